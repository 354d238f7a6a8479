"""Typed configuration of the Lunerax design, read from its own config.json keys.

A Lunerax config.json names the design in ``architecture`` and describes every layer in ``layers``: the kind of its
mixer (``type``: ``channel_delta``, ``latent_attention`` or ``attention``), the mixer's sizes and constants (``mixer``)
and its feed-forward (``mlp``: ``dense`` or null).  ``embedding.scale`` multiplies the embedded rows, ``norm.eps`` is
the constant of every norm, ``token_side.dim`` the width of what every token brings to every layer beside the stream,
and ``logit_softcap`` the cap of the logits.  Every size and constant comes from here; what the file does not mention
is not there (no window, no kept first tokens, no cap, no value mixing, no second embedding, no feed-forward).
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional, Tuple, Union

from .famepel_config import Rotation
from .model_config import ConfigError
from .mogisun_config import _need, _positive, _positive_int


def _optional_positive(d, key, where) -> Optional[float]:
    v = d.get(key)
    return None if v is None else _positive(v, f"{where}.{key}")


def _window(d, where) -> Tuple[Optional[int], int]:
    """(window or None, number of first tokens that stay visible behind it)."""
    mask = d.get("mask")
    if mask is None:
        return None, 0
    size = _positive_int(_need(mask, "size", f"{where}.mask"), f"{where}.mask.size")
    keep = mask.get("keep_first", 0)
    if isinstance(keep, bool) or not isinstance(keep, int) or keep < 0:
        raise ConfigError(f"{where}.mask.keep_first must be a count, got {keep!r}")
    return size, keep


def _grouped(heads, kv_heads, where):
    if heads % kv_heads:
        raise ConfigError(f"{where}: heads {heads} is not a multiple of kv_heads {kv_heads}")


@dataclass(frozen=True)
class ChannelDelta:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    decay_rank: Optional[int] = None     # ranks of the two low-rank pairs: from the checkpoint unless named
    gate_rank: Optional[int] = None

    @classmethod
    def from_dict(cls, d, where):
        m = cls(*(_positive_int(_need(d, k, where), f"{where}.{k}") for k in ("heads", "kv_heads", "dim", "vdim", "conv")),
                *(None if d.get(k) is None else _positive_int(d[k], f"{where}.{k}") for k in ("decay_rank", "gate_rank")))
        _grouped(m.heads, m.kv_heads, where)
        return m

    def to_dict(self) -> dict:
        d = {"conv": self.conv, "dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "vdim": self.vdim}
        d.update({k: v for k, v in (("decay_rank", self.decay_rank), ("gate_rank", self.gate_rank)) if v is not None})
        return d


@dataclass(frozen=True)
class LatentAttention:
    heads: int
    dim: int          # unrotated elements of a query or key head
    rot_dim: int      # rotated ones
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot: Rotation
    window: Optional[int] = None

    @classmethod
    def from_dict(cls, d, where):
        ints = [_positive_int(_need(d, k, where), f"{where}.{k}")
                for k in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank")]
        rot = Rotation.from_dict(_need(d, "rot", where), f"{where}.rot")
        if rot.dims > ints[2]:
            raise ConfigError(f"{where}: rot.dims {rot.dims} exceeds rot_dim {ints[2]}")
        if rot.scaling is not None:
            raise ConfigError(f"{where}.rot: this design does not stretch its frequencies")
        window, keep = _window(d, where)
        if keep:
            raise ConfigError(f"{where}.mask: latent attention keeps no first tokens")
        return cls(*ints, _positive(_need(d, "scale", where), f"{where}.scale"), rot, window)

    def to_dict(self) -> dict:
        d = {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank, "q_rank": self.q_rank,
             "rot": self.rot.to_dict(), "rot_dim": self.rot_dim, "scale": self.scale, "vdim": self.vdim}
        if self.window is not None:
            d["mask"] = {"size": self.window}
        return d


@dataclass(frozen=True)
class CappedAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: Optional[float] = None
    window: Optional[int] = None
    keep_first: int = 0
    v_mix: bool = False

    @classmethod
    def from_dict(cls, d, where):
        ints = [_positive_int(_need(d, k, where), f"{where}.{k}") for k in ("heads", "kv_heads", "dim", "vdim")]
        _grouped(ints[0], ints[1], where)
        v_mix = d.get("v_mix", False)
        if not isinstance(v_mix, bool):
            raise ConfigError(f"{where}.v_mix must be true or false, got {v_mix!r}")
        return cls(*ints, _positive(_need(d, "scale", where), f"{where}.scale"),
                   _optional_positive(d, "softcap", where), *_window(d, where), v_mix)

    def to_dict(self) -> dict:
        d = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale, "vdim": self.vdim,
             "v_mix": self.v_mix}
        if self.softcap is not None:
            d["softcap"] = self.softcap
        if self.window is not None:
            d["mask"] = {"keep_first": self.keep_first, "size": self.window}
        return d


@dataclass(frozen=True)
class DenseMlp:
    ff: int

    def to_dict(self) -> dict:
        return {"ff": self.ff, "kind": "dense"}


@dataclass(frozen=True)
class LuneraxLayer:
    type: str
    mixer: Union[ChannelDelta, LatentAttention, CappedAttention]
    mlp: Optional[DenseMlp]

    def to_dict(self) -> dict:
        return {"mixer": self.mixer.to_dict(), "mlp": self.mlp.to_dict() if self.mlp else None, "type": self.type}


_MIXERS = {"channel_delta": ChannelDelta, "latent_attention": LatentAttention, "attention": CappedAttention}


@dataclass(frozen=True)
class LuneraxConfig:
    vocab: int
    width: int
    norm_eps: float
    embedding_scale: float
    layers: Tuple[LuneraxLayer, ...]
    side_dim: Optional[int] = None
    logit_softcap: Optional[float] = None
    architecture: str = "Lunerax"

    @classmethod
    def from_dict(cls, d: Mapping[str, Any]) -> "LuneraxConfig":
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
                if _need(mlp, "kind", f"{where}.mlp") != "dense":
                    raise ConfigError(f"{where}.mlp.kind {mlp['kind']!r} is not implemented (known: 'dense')")
                mlp = DenseMlp(_positive_int(_need(mlp, "ff", f"{where}.mlp"), f"{where}.mlp.ff"))
            layers.append(LuneraxLayer(str(kind), mixer, mlp))
        mixing = [layer.mixer for layer in layers if isinstance(layer.mixer, CappedAttention) and layer.mixer.v_mix]
        if len({(m.kv_heads, m.vdim) for m in mixing}) > 1:
            raise ConfigError("layers that mix their values with the first one's have as many value heads of the same width")
        side = d.get("token_side")
        side_dim = None if side is None else _positive_int(_need(side, "dim", "token_side"), "token_side.dim")
        emb = d.get("embedding")
        scale = emb.get("scale", 1.0) if isinstance(emb, Mapping) else 1.0
        return cls(vocab, width, eps, _positive(scale, "embedding.scale"), tuple(layers), side_dim,
                   _optional_positive(d, "logit_softcap", "config"), str(d.get("architecture", "Lunerax")))

    def to_dict(self) -> dict:
        d = {"architecture": self.architecture, "embedding": {"scale": self.embedding_scale},
             "layers": [layer.to_dict() for layer in self.layers], "norm": {"eps": self.norm_eps},
             "vocab": self.vocab, "width": self.width}
        if self.side_dim is not None:
            d["token_side"] = {"dim": self.side_dim}
        if self.logit_softcap is not None:
            d["logit_softcap"] = self.logit_softcap
        return d
