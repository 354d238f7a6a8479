"""Token embedding and output head (reference: ``ops/embedding.py:49-92``).

The embedding gathers rows of ``[V, H]`` into the float32 residual, multiplied by ``scale`` if its params give one
(the product is taken in float32 on the stored row).  The head is
``logits = h E^T``; tied, it uses the embedding's storage (reference:
``ops/embedding.py:78-86``); untied, it has a matrix of its own, which the
reference mishandles by overwriting the embedding (``model/llama.py:147-154``).
With ``pairs`` (``{"buckets": B, "mul_prev": p, "mul_cur": c}``) the embedding adds a row of a second table ``[B + 1, H]``,
picked by the token ``t`` and the one before it, ``s``: row ``(s p + t c) mod B``, and row ``B`` for a sequence's first
token.  A sequence's last token is then state: one integer in the request's slot, which the kernel reads for a step's
first token and leaves holding the step's last.

Logits leave the head as float32; a head with a ``scale`` multiplies them by it, and one with a ``softcap`` ``c``
then maps every logit ``z`` to ``c * tanh(z / c)``.
"""

from __future__ import annotations

from .plan import StateNeed, TensorSpec
from .registry import register_embedding, register_head


@register_embedding("embedding")
class TokenEmbedding:
    """params: vocab_size, hidden_size, and optionally scale (every gathered row is multiplied by it) and pairs
    ({"buckets", "mul_prev", "mul_cur"}: a second table, picked by pairs of tokens)."""

    def __init__(self, params, env):
        self.vocab = int(params["vocab_size"])
        self.hidden = int(params["hidden_size"])
        self.scale = float(params.get("scale", 1.0))
        pairs = params.get("pairs")
        self.pairs = (int(pairs["buckets"]), int(pairs["mul_prev"]), int(pairs["mul_cur"])) if pairs else None
        if self.pairs is not None and (self.pairs[0] <= 0 or min(self.pairs[1:]) < 0 or max(self.pairs[1:]) >= 1 << 31):
            raise ValueError(f"pairs of tokens fall into a positive number of buckets by factors below 2^31, got {pairs}")
        self.env = env
        self.weight = self.pair_table = None

    def weight_specs(self):
        specs = {"weight": TensorSpec((self.vocab, self.hidden))}
        if self.pairs is not None:
            specs["pairs"] = TensorSpec((self.pairs[0] + 1, self.hidden))
        return specs

    def bind(self, tensors):
        self.weight = tensors["weight"]
        self.pair_table = tensors.get("pairs")

    def state_need(self):
        return StateNeed((1,), "int32", 0) if self.pairs is not None else None

    def forward(self, ctx, cache=None):
        if self.pairs is not None:
            return self.env.kernels.embed_pairs(ctx.token_ids, self.weight, self.pair_table, self.pairs, ctx, cache.state,
                                                scale=self.scale)
        if self.scale != 1.0:
            return self.env.kernels.embed(ctx.token_ids, self.weight, scale=self.scale)
        return self.env.kernels.embed(ctx.token_ids, self.weight)


@register_head("head")
class OutputHead:
    """params: vocab_size, hidden_size, tied, and optionally scale and softcap."""

    def __init__(self, params, env):
        self.vocab = int(params["vocab_size"])
        self.hidden = int(params["hidden_size"])
        self.tied = bool(params["tied"])
        self.scale = float(params.get("scale") or 1.0)
        self.softcap = float(params["softcap"]) if params.get("softcap") else None
        if self.softcap is not None and not self.softcap > 0:
            raise ValueError(f"a soft cap must be positive, got {self.softcap}")
        self.env = env
        self.embedding = None
        self._weight = None

    def share_embedding(self, embedding) -> None:
        """A tied head multiplies by the embedding's matrix: the same storage, not a copy."""
        if (embedding.vocab, embedding.hidden) != (self.vocab, self.hidden):
            raise ValueError(f"a head of {self.vocab} x {self.hidden} cannot share an embedding of "
                             f"{embedding.vocab} x {embedding.hidden}")
        self.embedding = embedding

    def weight_specs(self):
        return {} if self.tied else {"weight": TensorSpec((self.vocab, self.hidden))}

    def bind(self, tensors):
        if not self.tied:
            self._weight = tensors["weight"]
        elif self.embedding is None:
            raise ValueError("a tied head was given no embedding to share")

    @property
    def weight(self):
        return self.embedding.weight if self.tied else self._weight

    def forward(self, h):
        logits = self.env.kernels.linear(h, self.weight, out_float32=True)
        if self.scale != 1.0 or self.softcap is not None:
            logits = self.env.kernels.scale_softcap(logits, self.scale, self.softcap)
        return logits
