"""What a layer adds to the stream for the token itself, beside what the token's embedding started the stream with.

``gated_embedding``: a second embedding table holds a row for every token, cut into one part of ``dim`` elements per
layer.  A layer lets the stream decide how much of its part comes through:

    z = act(G x) * e            G [dim, hidden]; e = table[token, first_column : first_column + dim]
    y = P z                     P [hidden, dim]

``x`` is the residual stream in the compute dtype; the activation and the product with ``e`` are taken in float32 on the
product's sums where a kernel does both (few rows), and rounded once.  The norm on ``y`` is a part of its own.
"""

from __future__ import annotations

import torch

from .dense import ACTIVATIONS
from .plan import TensorSpec
from .registry import register_token_input


@register_token_input("gated_embedding")
class GatedEmbedding:
    """params: hidden_size, vocab_size, dim, first_column, table_width, activation."""

    def __init__(self, params, env):
        self.hidden = int(params["hidden_size"])
        self.vocab = int(params["vocab_size"])
        self.dim = int(params["dim"])
        self.first_column = int(params["first_column"])
        self.table_width = int(params["table_width"])
        self.activation = str(params["activation"])
        if self.activation not in ACTIVATIONS:
            raise ValueError(f"activation {self.activation!r} is not one of {', '.join(ACTIVATIONS)}")
        if not 0 <= self.first_column <= self.table_width - self.dim:
            raise ValueError(f"columns {self.first_column} .. {self.first_column + self.dim} lie outside a table row of "
                             f"{self.table_width}")
        self.env = env
        self.table = self.w_gate = self.w_proj = None

    def weight_specs(self):
        return {"table": TensorSpec((self.vocab, self.table_width)), "gate": TensorSpec((self.dim, self.hidden)),
                "proj": TensorSpec((self.hidden, self.dim))}

    def bind(self, tensors):
        self.table = tensors["table"]       # the same tensor for every layer
        self.w_gate, self.w_proj = tensors["gate"].contiguous(), tensors["proj"].contiguous()
        pad = -self.dim % 64 if self.w_proj.dtype == torch.bfloat16 else 0
        if pad:     # the few-row product wants its inner size a multiple of 64: zero columns, and as many zeros of z
            self.w_gate = torch.cat([self.w_gate, self.w_gate.new_zeros((pad, self.hidden))]).contiguous()
            self.w_proj = torch.cat([self.w_proj, self.w_proj.new_zeros((self.hidden, pad))], dim=1).contiguous()

    def forward(self, x, ctx):
        k = self.env.kernels
        z = k.embedding_gate(x, self.w_gate, self.activation, self.table, self.first_column, self.dim, ctx.token_ids)
        return k.linear(z, self.w_proj)
