"""Dense gated feed-forward (reference: ``ops/mlp.py:87-128``).

``y = (silu(h Wg^T) * (h Wu^T)) Wd^T``.  Gate and up are stacked into one
``[2I, H]`` matrix at load (reference: ``ops/mlp.py:104``) so one product gives
both; ``silu(g) * u`` is computed in float32 and rounded once (reference:
``kernels/swiglu_kernel.py:142-150``).  With ``activation: "relu"`` the gate is ``max(g, 0) * u`` instead,
with ``"gelu_tanh"`` it is ``gelu(g) * u`` in the tanh form.  With ``bias`` all three projections have biases: those of gate and
up are added to the product's sums in front of the activation, that of down goes on with the result (``BiasedDelta``).
"""

from __future__ import annotations

import torch

from .context import BiasedDelta
from .plan import TensorSpec
from .registry import register_feed_forward


@register_feed_forward("swiglu")
class SwiGLU:
    """params: hidden_size, intermediate_size, and optionally activation ("silu", the default, "relu" or "gelu_tanh") and
    bias (default False)."""

    takes_scaled_rows = True   # the input goes to ``gated_linear`` only

    def __init__(self, params, env):
        self.hidden = int(params["hidden_size"])
        self.inter = int(params["intermediate_size"])
        self.activation = str(params.get("activation", "silu"))
        if self.activation not in ("silu", "relu", "gelu_tanh"):
            raise ValueError(f"a gated feed-forward's activation is silu, relu or gelu_tanh, not {self.activation!r}")
        self.bias = bool(params.get("bias", False))
        if self.bias and self.activation == "silu":
            raise ValueError("the silu gate has no biases")
        self.b_gate_up = self.b_down = None
        self.env = env
        self.w_gate_up = None
        self.w_down = None

    def weight_specs(self):
        specs = {
            "gate": TensorSpec((self.inter, self.hidden)),
            "up": TensorSpec((self.inter, self.hidden)),
            "down": TensorSpec((self.hidden, self.inter)),
        }
        if self.bias:
            specs.update({"gate_bias": TensorSpec((self.inter,), "vector"), "up_bias": TensorSpec((self.inter,), "vector"),
                          "down_bias": TensorSpec((self.hidden,), "vector")})
        return specs

    def bind(self, tensors):
        self.w_gate_up = torch.cat([tensors["gate"], tensors["up"]], dim=0).contiguous()
        self.w_down = tensors["down"].contiguous()
        if self.bias:
            self.b_gate_up = torch.cat([tensors["gate_bias"], tensors["up_bias"]]).float().contiguous()
            self.b_down = tensors["down_bias"].contiguous()
        prepare = getattr(self.env.kernels, "prepare_pending_weight", None)
        if prepare is not None:   # the kernels may keep a copy of their own of a weight whose product is left pending
            prepare(self.w_down)

    def plain_form(self):
        """What this feed-forward is, as plain data, for kernels that can run a whole block in one call (None for
        a subclass with a forward of its own: it is no longer what this form describes)."""
        if type(self).forward is not SwiGLU.forward or self.activation != "silu":
            return None
        return {"kind": "swiglu", "w_gate_up": self.w_gate_up, "w_down": self.w_down, "hidden": self.hidden,
                "inter": self.inter}

    def forward(self, h, ctx):
        k = self.env.kernels
        if self.activation == "silu":
            a = k.gated_linear(h, self.w_gate_up)   # the activation is fused into the product where a kernel has it
        else:
            a = k.gated_linear(h, self.w_gate_up, activation=(self.activation, None), bias=self.b_gate_up) if self.bias \
                else k.gated_linear(h, self.w_gate_up, activation=(self.activation, None))
        if self.bias:
            return BiasedDelta(k.pending_linear(a, self.w_down), self.b_down, k)
        return k.pending_linear(a, self.w_down)   # the norm after it may have it added into the residual
