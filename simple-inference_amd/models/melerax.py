"""``Melerax``: a decoder with its norms behind the sublayers, whose mixers are attention inside blocks of positions
beside a gated linear recurrent unit, a matrix state with a bonus for the current token, and the recurrent unit alone.

All that is particular to the design is here: which parts a layer has and what the tensors are called.

* A layer is an output-norm block: ``x += N1(mixer(x)) * s1`` and, if it has a feed-forward, ``x += N2(ff(x)) * s2``;
  every ``N`` is an RMS norm whose gain is stored as its distance from one, ``s`` a stored vector.
* ``parallel``: ``parts/parallel.py`` over the ``attention`` part (biases, a short convolution on q, k and v, a norm over
  the whole rows of q and k, neighbouring elements rotated, capped scores, blocks of positions) and the ``rglru`` part;
  half the sum of the two results, each behind an RMS norm of its own.
* ``wkv``: ``parts/wkv.py``.  ``rglru``: ``parts/rglru.py``.
* ``dense``: ``W_down (gelu(W_gate h + b) * (W_up h + b)) + b`` with the tanh form of the gelu.  ``moe``: experts
  ``W_down gelu(W_up h)`` with the exact gelu, chosen by the largest biased router logits and weighted by the softmax over
  these; a shared expert of the same form.
* The embedding adds a row of a table of token pairs; the last norm is of the layers' kind; the head is untied.

Checkpoint names: ``embed``, ``bigram``, ``final.norm``, ``head``; layer ``i``: ``l<i>.norm1``, ``l<i>.norm2``,
``l<i>.ls1``, ``l<i>.ls2``, ``l<i>.mix.*`` (under ``.left`` and ``.right`` for mixers side by side), ``l<i>.mlp.*``; a bias
has its weight's name with ``.b`` added.
"""

from __future__ import annotations

from ..config.lunerax_config import DenseMlp
from ..config.melerax_config import LinearUnit, MeleraxConfig, ParallelMixer, PlainExperts, WkvMixer
from ..config.registry import register_architecture
from ..parts.plan import LayerSpec, ModelPlan, PartSpec


def _linear_unit(cfg: MeleraxConfig, m: LinearUnit, p: str):
    names = {n: f"{p}.{n}" for n in ("y", "x", "conv", "ra", "ri", "lam", "o")}
    names.update({f"{n}_bias": f"{p}.{n}.b" for n in ("y", "x", "conv", "ra", "ri")})
    return {"hidden_size": cfg.width, "width": m.width, "blocks": m.blocks, "conv_taps": m.conv}, names


def _mixer(cfg: MeleraxConfig, m, p: str) -> PartSpec:
    if isinstance(m, WkvMixer):
        names = {n: f"{p}.{n}" for n in ("r", "k", "v", "g", "w1", "w2", "w0", "u", "norm", "o")}
        names.update({f"mu_{n}": f"{p}.mu.{n}" for n in "rkvgw"})
        return PartSpec("wkv", {"hidden_size": cfg.width, "num_heads": m.heads, "head_dim": m.dim,
                                "norm_eps": cfg.norm_eps, "decay_rank": m.decay_rank}, names, role="mixer")
    if isinstance(m, LinearUnit):
        params, names = _linear_unit(cfg, m, p)
        return PartSpec("rglru", params, names, role="mixer")
    assert isinstance(m, ParallelMixer)
    left = m.left
    position = {"kind": "none", "params": {}}
    if left.rot is not None:
        position = {"kind": "rope", "params": {"rotary_dim": left.rot.dims, "theta": left.rot.base, "scaling": None,
                                               "pairing": "interleaved", "angles": "float64"}}
    right, right_names = _linear_unit(cfg, m.right, f"{p}.right")
    norm = {"eps": cfg.norm_eps}
    branches = {
        "left": {"kind": "attention", "scale": 0.5, "norm": norm, "params": {
            "hidden_size": cfg.width, "num_heads": left.heads, "num_kv_heads": left.kv_heads, "head_dim": left.dim,
            "value_head_dim": left.vdim, "scale": left.scale, "softcap": left.softcap, "chunk": left.block, "bias": True,
            "conv_taps": left.conv, "qk_norm": {"eps": cfg.norm_eps, "over": "row"}, "position": position}},
        "right": {"kind": "rglru", "scale": 0.5, "norm": norm, "params": right},
    }
    names = {f"left.{n}": f"{p}.left.{n}" for n in ("q", "k", "v", "o")}
    names.update({f"left.{n}_bias": f"{p}.left.{n}.b" for n in "qkv"})
    names.update({f"left.{n}_conv": f"{p}.left.{n}.conv" for n in "qkv"})
    names.update({f"left.{n}_norm": f"{p}.left.{n}.norm" for n in "qk"})
    names.update({f"right.{n}": name for n, name in right_names.items()})
    names.update({f"{side}.result_norm": f"{p}.{side}.out" for side in branches})
    return PartSpec("parallel", {"branches": branches}, names, role="mixer")


def _feed_forward(cfg: MeleraxConfig, mlp, p: str) -> PartSpec:
    if isinstance(mlp, DenseMlp):
        names = {n: f"{p}.{n}" for n in ("gate", "up", "down")}
        names.update({f"{n}_bias": f"{p}.{n}.b" for n in ("gate", "up", "down")})
        return PartSpec("swiglu", {"hidden_size": cfg.width, "intermediate_size": mlp.ff, "activation": "gelu_tanh",
                                   "bias": True}, names, role="feed_forward")
    assert isinstance(mlp, PlainExperts)
    names = {"router": f"{p}.router", "router_bias": f"{p}.router.b"}
    for e in range(mlp.experts):
        names.update({f"up{e}": f"{p}.e{e}.up", f"down{e}": f"{p}.e{e}.down"})
    params = {"hidden_size": cfg.width, "experts": mlp.experts, "top": mlp.top, "expert_size": mlp.ff,
              "activation": "gelu", "router_bias": True}
    if mlp.shared_ff is not None:
        params.update({"shared_size": mlp.shared_ff, "shared_gate": False})
        names.update({"shared_up": f"{p}.shared.up", "shared_down": f"{p}.shared.down"})
    return PartSpec("moe", params, names, role="feed_forward")


def melerax_plan(cfg: MeleraxConfig) -> ModelPlan:
    def norm(name, scale=None, role="norm"):
        params = {"size": cfg.width, "eps": cfg.norm_eps, "unit_offset": True, "scaled": scale is not None}
        return PartSpec("rmsnorm", params, {"weight": name, **({"scale": scale} if scale else {})}, role=role)

    layers = []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}"
        parts = {"mixer": _mixer(cfg, layer.mixer, f"{p}.mix"), "mixer_norm": norm(f"{p}.norm1", f"{p}.ls1")}
        if layer.mlp is not None:
            parts.update({"feed_forward": _feed_forward(cfg, layer.mlp, f"{p}.mlp"),
                          "feed_forward_norm": norm(f"{p}.norm2", f"{p}.ls2")})
        layers.append(LayerSpec(block="output_norm", parts=parts))
    embedding = {"vocab_size": cfg.vocab, "hidden_size": cfg.width}
    names = {"weight": "embed"}
    if cfg.bigram is not None:
        embedding["pairs"] = cfg.bigram.to_dict()
        names["pairs"] = "bigram"
    return ModelPlan(
        hidden_size=cfg.width,
        vocab_size=cfg.vocab,
        embedding=PartSpec("embedding", embedding, names),
        layers=layers,
        final_norm=norm("final.norm", role=""),
        head=PartSpec("head", {"vocab_size": cfg.vocab, "hidden_size": cfg.width, "tied": False}, {"weight": "head"}),
    )


register_architecture("Melerax", MeleraxConfig.from_dict, melerax_plan, replace=True)
