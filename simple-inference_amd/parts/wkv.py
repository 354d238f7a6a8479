"""A matrix state per head with a decay per key channel and a bonus for the current token (the RWKV form).

For a token with input ``h`` and the token before it, ``h'`` (zeros before the first), ``H`` heads of width ``D``:

    m_s = h + (h' - h) * mu_s                             for each s of r, k, v, g, w
    r, k, v = W_r m_r, W_k m_k, W_v m_v                   [H, D]
    w = exp(-exp(W_2 tanh(W_1 m_w) + w0))                 [H, D], through a low-rank pair
    o = (S + diag(u) k v^T)^T r;   S <- diag(w) S + k v^T            S [D, D]
    y = W_o (concat(o_h / rms(o_h)) * n * silu(W_g m_g))             n [H D]

A request's row of state holds, in float32, the ``H`` matrices and behind them the last token's ``h``.  The five input
products share one stacked matrix whose groups of rows read inputs of their own.  Decays, the state, the norm and the
gate's product are float32 in both modes.  The rank of the low-rank pair is whatever the checkpoint's tensors have, unless
``decay_rank`` names it.
"""

from __future__ import annotations

import torch

from .plan import StateNeed, TensorSpec
from .registry import register_mixer

SHIFTED = ("r", "k", "v", "g", "w")


@register_mixer("wkv")
class WkvMixer:
    """params: hidden_size, num_heads, head_dim, norm_eps, and optionally decay_rank."""

    def __init__(self, params, env):
        self.hidden = int(params["hidden_size"])
        self.num_heads = int(params["num_heads"])
        self.head_dim = int(params["head_dim"])
        self.eps = float(params["norm_eps"])
        rank = params.get("decay_rank")
        self.rank = int(rank) if rank else -1
        self.inner = self.num_heads * self.head_dim
        check = getattr(env.kernels, "check_recurrent_geometry", None)
        if check is not None:
            check(self.head_dim, self.head_dim)
        self.env = env
        self.w_in = self.w_o = self.mu = self.w2 = self.w0 = self.u = self.norm = None

    takes_scaled_rows = False

    def weight_specs(self):
        inner = self.inner
        specs = {f"mu_{s}": TensorSpec((self.hidden,), "vector") for s in SHIFTED}
        specs.update({s: TensorSpec((inner, self.hidden)) for s in "rkvg"})
        specs.update({"w1": TensorSpec((self.rank, self.hidden)), "w2": TensorSpec((inner, self.rank)),
                      "w0": TensorSpec((inner,), "vector"), "u": TensorSpec((self.num_heads, self.head_dim), "vector"),
                      "norm": TensorSpec((inner,), "vector"), "o": TensorSpec((self.hidden, inner))})
        return specs

    def bind(self, tensors):
        rank, second = tensors["w1"].shape[0], tensors["w2"].shape[1]
        if rank != second or (self.rank > 0 and rank != self.rank):
            raise ValueError(f"the decay's low-rank pair does not fit: w1 gives {rank} columns, w2 takes {second}"
                             f"{f', expected {self.rank}' if self.rank > 0 else ''}")
        self.mu = torch.stack([tensors[f"mu_{s}"].float() for s in SHIFTED]).contiguous()
        self.w_in = torch.cat([tensors[s] for s in ("r", "k", "v", "g", "w1")], dim=0).contiguous()
        self.w2, self.w_o = tensors["w2"].contiguous(), tensors["o"].contiguous()
        self.w0, self.norm = tensors["w0"].float().contiguous(), tensors["norm"].float().contiguous()
        self.u = tensors["u"].float().reshape(-1).contiguous()
        prepare = getattr(self.env.kernels, "prepare_pending_weight", None)
        if prepare is not None:
            prepare(self.w_o)

    def cache_need(self):
        return None

    @property
    def matrix_floats(self) -> int:
        return self.num_heads * self.head_dim * self.head_dim

    def state_need(self):
        return StateNeed((self.matrix_floats + self.hidden,), "float32", 0.0)

    def forward(self, h, ctx, cache):
        k = self.env.kernels
        mixed = k.token_shift(h, self.mu, ctx, cache.state, self.matrix_floats)
        rkvg, low = k.grouped_linear(mixed, self.w_in, self.inner)
        out = k.bonus_recurrence(rkvg, low, self.w2, self.w0, self.u, self.norm, self.num_heads, self.head_dim, self.eps,
                                 ctx, cache.state)
        return k.pending_linear(out, self.w_o)
