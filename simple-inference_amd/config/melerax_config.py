"""Typed configuration of the Melerax design, read from its own config.json keys.

A Melerax config.json names the design in ``architecture`` and describes every layer in ``layers``: the kind of its
mixer (``type``: ``parallel``, ``wkv`` or ``rglru``), the mixer's sizes and constants (``mixer``) and its feed-forward
(``mlp``: ``dense``, ``moe`` or null).  ``embedding.bigram`` sizes the table of token pairs and the hash that picks its
rows, ``norm.eps`` is the constant of every norm.  Every size and constant comes from here; what the file does not
mention is not there (no pair table, no block mask, no cap, no rotation, no shared expert, no feed-forward).  The rank of
the decay's low-rank pair has no key of its own and is read from the checkpoint unless ``decay_rank`` names it.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional, Tuple, Union

from .famepel_config import Rotation
from .lunerax_config import DenseMlp, _grouped, _optional_positive
from .model_config import ConfigError
from .mogisun_config import _need, _positive, _positive_int


@dataclass(frozen=True)
class BlockAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    scale: float
    rot: Optional[Rotation] = None
    softcap: Optional[float] = None
    block: Optional[int] = None      # positions of a block inside which a query attends

    @classmethod
    def from_dict(cls, d, where):
        ints = [_positive_int(_need(d, k, where), f"{where}.{k}") for k in ("heads", "kv_heads", "dim", "vdim", "conv")]
        _grouped(ints[0], ints[1], where)
        rot = None
        if d.get("rot") is not None:
            rot = Rotation.from_dict(d["rot"], f"{where}.rot")
            if rot.dims > ints[2]:
                raise ConfigError(f"{where}: rot.dims {rot.dims} exceeds dim {ints[2]}")
            if rot.scaling is not None:
                raise ConfigError(f"{where}.rot: this design does not stretch its frequencies")
        mask = d.get("mask")
        block = None if mask is None else _positive_int(_need(mask, "size", f"{where}.mask"), f"{where}.mask.size")
        return cls(*ints, _positive(_need(d, "scale", where), f"{where}.scale"), rot,
                   _optional_positive(d, "softcap", where), block)

    def to_dict(self) -> dict:
        d = {"conv": self.conv, "dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale,
             "vdim": self.vdim}
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        if self.softcap is not None:
            d["softcap"] = self.softcap
        if self.block is not None:
            d["mask"] = {"size": self.block}
        return d


@dataclass(frozen=True)
class LinearUnit:
    width: int
    blocks: int
    conv: int

    @classmethod
    def from_dict(cls, d, where):
        m = cls(*(_positive_int(_need(d, k, where), f"{where}.{k}") for k in ("width", "blocks", "conv")))
        if m.width % m.blocks:
            raise ConfigError(f"{where}: width {m.width} does not split into {m.blocks} equal blocks")
        return m

    def to_dict(self) -> dict:
        return {"blocks": self.blocks, "conv": self.conv, "width": self.width}


@dataclass(frozen=True)
class ParallelMixer:
    left: BlockAttention
    right: LinearUnit

    @classmethod
    def from_dict(cls, d, where):
        return cls(BlockAttention.from_dict(_need(d, "left", where), f"{where}.left"),
                   LinearUnit.from_dict(_need(d, "right", where), f"{where}.right"))

    def to_dict(self) -> dict:
        return {"left": self.left.to_dict(), "right": self.right.to_dict()}


@dataclass(frozen=True)
class WkvMixer:
    heads: int
    dim: int
    decay_rank: Optional[int] = None

    @classmethod
    def from_dict(cls, d, where):
        return cls(*(_positive_int(_need(d, k, where), f"{where}.{k}") for k in ("heads", "dim")),
                   None if d.get("decay_rank") is None else _positive_int(d["decay_rank"], f"{where}.decay_rank"))

    def to_dict(self) -> dict:
        d = {"dim": self.dim, "heads": self.heads}
        if self.decay_rank is not None:
            d["decay_rank"] = self.decay_rank
        return d


@dataclass(frozen=True)
class PlainExperts:
    """Experts without a gate, chosen by biased router logits."""

    experts: int
    top: int
    ff: int
    shared_ff: Optional[int] = None

    @classmethod
    def from_dict(cls, d, where):
        router = _need(d, "router", where)
        experts = _positive_int(_need(router, "experts", f"{where}.router"), f"{where}.router.experts")
        top = _positive_int(_need(router, "top", f"{where}.router"), f"{where}.router.top")
        if top > experts:
            raise ConfigError(f"{where}.router: top {top} exceeds the number of experts {experts}")
        ff = _positive_int(_need(_need(d, "expert", where), "ff", f"{where}.expert"), f"{where}.expert.ff")
        shared = d.get("shared")
        return cls(experts, top, ff,
                   None if shared is None else _positive_int(_need(shared, "ff", f"{where}.shared"), f"{where}.shared.ff"))

    def to_dict(self) -> dict:
        d = {"expert": {"ff": self.ff}, "kind": "moe", "router": {"experts": self.experts, "top": self.top}}
        if self.shared_ff is not None:
            d["shared"] = {"ff": self.shared_ff}
        return d


@dataclass(frozen=True)
class MeleraxLayer:
    type: str
    mixer: Union[ParallelMixer, WkvMixer, LinearUnit]
    mlp: Optional[Union[DenseMlp, PlainExperts]]

    def to_dict(self) -> dict:
        return {"mixer": self.mixer.to_dict(), "mlp": self.mlp.to_dict() if self.mlp else None, "type": self.type}


@dataclass(frozen=True)
class Bigram:
    """A table of ``buckets + 1`` rows; a token behind another takes row ``(previous * mul_prev + token * mul_cur) mod
    buckets``, a sequence's first token the last row."""

    buckets: int
    mul_prev: int
    mul_cur: int

    @classmethod
    def from_dict(cls, d, where):
        muls = []
        for k in ("mul_prev", "mul_cur"):
            v = _need(d, k, where)
            if isinstance(v, bool) or not isinstance(v, int) or not 0 <= v < 1 << 31:
                raise ConfigError(f"{where}.{k} must be an integer from 0 to 2^31 - 1, got {v!r}")
            muls.append(v)
        return cls(_positive_int(_need(d, "buckets", where), f"{where}.buckets"), *muls)

    def to_dict(self) -> dict:
        return {"buckets": self.buckets, "mul_cur": self.mul_cur, "mul_prev": self.mul_prev}


_MIXERS = {"parallel": ParallelMixer, "wkv": WkvMixer, "rglru": LinearUnit}


@dataclass(frozen=True)
class MeleraxConfig:
    vocab: int
    width: int
    norm_eps: float
    layers: Tuple[MeleraxLayer, ...]
    bigram: Optional[Bigram] = None
    architecture: str = "Melerax"

    @classmethod
    def from_dict(cls, d: Mapping[str, Any]) -> "MeleraxConfig":
        vocab = _positive_int(_need(d, "vocab", "config"), "vocab")
        width = _positive_int(_need(d, "width", "config"), "width")
        eps = _positive(_need(_need(d, "norm", "config"), "eps", "norm"), "norm.eps")
        entries = _need(d, "layers", "config")
        if not isinstance(entries, (list, tuple)) or not entries:
            raise ConfigError("config.json's layers must be a list with at least one layer")
        layers = []
        for i, e in enumerate(entries):
            where = f"layers[{i}]"
            kind = _need(e, "type", where)
            if kind not in _MIXERS:
                raise ConfigError(f"{where}.type {kind!r} is not implemented (known: {', '.join(sorted(_MIXERS))})")
            mixer = _MIXERS[kind].from_dict(_need(e, "mixer", where), f"{where}.mixer")
            mlp = e.get("mlp")
            if mlp is not None:
                form = _need(mlp, "kind", f"{where}.mlp")
                if form == "dense":
                    mlp = DenseMlp(_positive_int(_need(mlp, "ff", f"{where}.mlp"), f"{where}.mlp.ff"))
                elif form == "moe":
                    mlp = PlainExperts.from_dict(mlp, f"{where}.mlp")
                else:
                    raise ConfigError(f"{where}.mlp.kind {form!r} is not implemented (known: 'dense', 'moe')")
            layers.append(MeleraxLayer(str(kind), mixer, mlp))
        bigram = (d.get("embedding") or {}).get("bigram")
        return cls(vocab, width, eps, tuple(layers),
                   None if bigram is None else Bigram.from_dict(bigram, "embedding.bigram"),
                   str(d.get("architecture", "Melerax")))

    def to_dict(self) -> dict:
        d = {"architecture": self.architecture, "layers": [layer.to_dict() for layer in self.layers],
             "norm": {"eps": self.norm_eps}, "vocab": self.vocab, "width": self.width}
        if self.bigram is not None:
            d["embedding"] = {"bigram": self.bigram.to_dict()}
        return d
