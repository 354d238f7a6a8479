"""The recurrent block of a real-gated linear recurrent unit: a diagonal recurrence whose decay the input decides.

For a token with input ``h`` (inner width ``W``, cut into ``blocks`` equal parts):

    y = gelu(W_y h + b_y)                                 tanh form
    u = conv(W_x h + b_x) + c                             a short causal convolution per channel, no activation
    r = sigmoid(R_b u_b + rb_b),  i = sigmoid(I_b u_b + ib_b)      per part b, square matrices
    log a = -8 r softplus(lam)
    S <- a S + sqrt(1 - a^2) i u                          [W], from zero, the first token included
    out = W_o (S * y)

A request's row of state holds, in float32, ``S`` and behind it the last inputs of the convolution as a ring: the input
of position ``p`` lies in ring row ``p mod taps``, so that a step's single token writes a row that no thread reads.  The two
input projections are one stacked matrix ``[y | x]``.  Gates, decays and the state are float32 in both modes.
"""

from __future__ import annotations

import torch

from .plan import StateNeed, TensorSpec
from .registry import register_mixer

RATE = 8.0     # the constant in front of the gate in the decay's logarithm


@register_mixer("rglru")
class LinearRecurrentUnit:
    """params: hidden_size, width, blocks, conv_taps."""

    def __init__(self, params, env):
        self.hidden = int(params["hidden_size"])
        self.width = int(params["width"])
        self.blocks = int(params["blocks"])
        self.taps = int(params["conv_taps"])
        if self.blocks < 1 or self.width % self.blocks or self.taps < 1:
            raise ValueError(f"a width of {self.width} does not split into {self.blocks} equal parts (or the convolution "
                             f"has no tap)")
        self.block = self.width // self.blocks
        check = getattr(env.kernels, "check_linear_unit", None)
        if check is not None:
            check(self.block, self.taps)
        self.env = env
        self.w_in = self.w_o = None
        self.terms = None
        self.x_col = self.width + (-self.width) % 8      # each part of a projected row starts aligned

    takes_scaled_rows = False
    takes_projection = True       # ``forward_projected`` may be handed the rows of ``w_in``'s product

    def weight_specs(self):
        W, bs = self.width, self.block
        vector = lambda *shape: TensorSpec(shape, "vector")
        return {"y": TensorSpec((W, self.hidden)), "y_bias": vector(W), "x": TensorSpec((W, self.hidden)), "x_bias": vector(W),
                "conv": vector(W, self.taps), "conv_bias": vector(W), "ra": TensorSpec((self.blocks, bs, bs)),
                "ra_bias": vector(self.blocks, bs), "ri": TensorSpec((self.blocks, bs, bs)), "ri_bias": vector(self.blocks, bs),
                "lam": vector(W), "o": TensorSpec((self.hidden, W))}

    def bind(self, tensors):
        gap = lambda t: [t.new_zeros((-self.width % 8, self.hidden))] if self.width % 8 else []
        self.w_in = torch.cat([tensors["y"], *gap(tensors["y"]), tensors["x"], *gap(tensors["x"])], dim=0).contiguous()
        self.w_o = tensors["o"].contiguous()
        f32 = lambda n: tensors[n].float().reshape(-1).contiguous()
        self.terms = {
            "y_bias": f32("y_bias"), "x_bias": f32("x_bias"), "conv": tensors["conv"].float().t().contiguous(),
            "conv_bias": f32("conv_bias"), "ra": tensors["ra"].contiguous(), "ri": tensors["ri"].contiguous(),
            "ra_bias": f32("ra_bias"), "ri_bias": f32("ri_bias"),
            "rate": RATE * torch.nn.functional.softplus(tensors["lam"].double(), threshold=1e9).float().contiguous(),
        }
        prepare = getattr(self.env.kernels, "prepare_pending_weight", None)
        if prepare is not None:
            prepare(self.w_o)

    def cache_need(self):
        return None

    def state_need(self):
        return StateNeed((self.width * (1 + (self.taps if self.taps > 1 else 0)),), "float32", 0.0)

    def forward(self, h, ctx, cache):
        return self.forward_projected(self.env.kernels.linear(h, self.w_in), ctx, cache)

    def forward_projected(self, proj, ctx, cache):
        k = self.env.kernels
        out = k.linear_unit(proj, 0, self.x_col, self.terms, self.blocks, ctx, cache.state)
        return k.pending_linear(out, self.w_o)
