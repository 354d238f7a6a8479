"""``Lunerax``: a pre-norm decoder whose every layer also takes something of the token itself, and whose mixers are a
delta rule with a decay per key channel, latent attention over a window, and attention without positions.

All that is particular to the design is here: which parts a layer has and what the tensors are called.

* A layer is a pre-norm block with a token input: ``x += mixer(L1(x))``, ``x += ff(L2(x))`` if it has a feed-forward,
  then ``x += rms(P (gelu(G x) * e)) * s`` with ``e`` the layer's part of the token's row of a second embedding; every
  ``L`` is a layer norm with weight and bias.
* ``channel_delta``: the delta rule of ``parts/delta.py`` with a decay for every key channel and a sigmoid output gate,
  both through low-rank pairs.
* ``latent_attention``: ``parts/latent_attention.py`` over a window, with a sigmoid gate on every element of the heads.
* ``attention``: ``parts/attention.py`` without a rotation; capped scores, a window that keeps the first tokens, values
  mixed with those of the first layer that mixes, the same gate.
* ``dense``: ``W_down (relu(W_gate h) * (W_up h))``.
* The embedding is multiplied by ``embedding.scale``; the last norm is a layer norm too; the head is untied and its
  logits are capped softly.

Checkpoint names: ``embed``, ``side.embed``, ``final.norm``, ``head``; layer ``i``: ``l<i>.norm1``, ``l<i>.norm2``,
``l<i>.mix.*``, ``l<i>.mlp.*``, ``l<i>.side.*``; a layer norm's bias has its weight's name with ``.b`` added.
"""

from __future__ import annotations

from ..config.lunerax_config import CappedAttention, ChannelDelta, LatentAttention, LuneraxConfig
from ..config.registry import register_architecture
from ..parts.plan import LayerSpec, ModelPlan, PartSpec


def _mixer(cfg: LuneraxConfig, i: int, first_mixing) -> PartSpec:
    m, p = cfg.layers[i].mixer, f"l{i}.mix"
    if isinstance(m, ChannelDelta):
        names = {n: f"{p}.{n}" for n in ("q", "k", "v", "b", "a1", "a2", "g1", "g2", "dt_bias", "norm", "o")}
        names.update({"q_conv": f"{p}.q.conv", "k_conv": f"{p}.k.conv", "v_conv": f"{p}.v.conv", "a_log": f"{p}.A_log"})
        return PartSpec("channel_delta", {
            "hidden_size": cfg.width, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "key_dim": m.dim,
            "value_dim": m.vdim, "conv_taps": m.conv, "norm_eps": cfg.norm_eps, "decay_rank": m.decay_rank,
            "gate_rank": m.gate_rank}, names, role="mixer")
    if isinstance(m, LatentAttention):
        names = {n: f"{p}.{n}" for n in ("dq", "uq", "dkv", "uk", "uv", "o")}
        names.update({"dq_norm": f"{p}.dq.norm", "dkv_norm": f"{p}.dkv.norm", "gate": f"{p}.g"})
        return PartSpec("latent_attention", {
            "hidden_size": cfg.width, "num_heads": m.heads, "head_dim": m.dim, "rot_dim": m.rot_dim,
            "value_head_dim": m.vdim, "q_rank": m.q_rank, "kv_rank": m.kv_rank, "scale": m.scale,
            "norm_eps": cfg.norm_eps, "window": m.window, "out_gate": "element",
            "position": {"kind": "rope", "params": {"rotary_dim": m.rot.dims, "theta": m.rot.base, "scaling": None,
                                                    "angles": "float64"}}}, names, role="mixer")
    assert isinstance(m, CappedAttention)
    names = {n: f"{p}.{n}" for n in ("q", "k", "v", "o")}
    names.update({"gate": f"{p}.g", "value_mix": f"{p}.vmix"})
    return PartSpec("attention", {
        "hidden_size": cfg.width, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim,
        "value_head_dim": m.vdim, "scale": m.scale, "softcap": m.softcap, "window": m.window,
        "keep_first": m.keep_first, "out_gate": "element",
        "value_mix": ("gives" if i == first_mixing else "takes") if m.v_mix else None,
        "position": {"kind": "none", "params": {}}}, names, role="mixer")


def lunerax_plan(cfg: LuneraxConfig) -> ModelPlan:
    def norm(name, role="norm"):
        return PartSpec("layernorm", {"size": cfg.width, "eps": cfg.norm_eps}, {"weight": name, "bias": name + ".b"}, role=role)

    first_mixing = next((i for i, layer in enumerate(cfg.layers)
                         if isinstance(layer.mixer, CappedAttention) and layer.mixer.v_mix), None)
    layers = []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}"
        parts = {"mixer_norm": norm(f"{p}.norm1"), "mixer": _mixer(cfg, i, first_mixing)}
        if layer.mlp is not None:
            parts["feed_forward_norm"] = norm(f"{p}.norm2")
            parts["feed_forward"] = PartSpec(
                "swiglu", {"hidden_size": cfg.width, "intermediate_size": layer.mlp.ff, "activation": "relu"},
                {n: f"{p}.mlp.{n}" for n in ("gate", "up", "down")}, role="feed_forward")
        if cfg.side_dim is not None:
            parts["token_input"] = PartSpec("gated_embedding", {
                "hidden_size": cfg.width, "vocab_size": cfg.vocab, "dim": cfg.side_dim, "first_column": i * cfg.side_dim,
                "table_width": len(cfg.layers) * cfg.side_dim, "activation": "gelu_tanh"},
                {"table": "side.embed", "gate": f"{p}.side.gate", "proj": f"{p}.side.proj"}, role="token_input")
            parts["token_input_norm"] = PartSpec("rmsnorm", {"size": cfg.width, "eps": cfg.norm_eps},
                                                 {"weight": f"{p}.side.norm"}, role="norm")
        layers.append(LayerSpec(block="prenorm", parts=parts))
    return ModelPlan(
        hidden_size=cfg.width,
        vocab_size=cfg.vocab,
        embedding=PartSpec("embedding", {"vocab_size": cfg.vocab, "hidden_size": cfg.width,
                                         "scale": cfg.embedding_scale}, {"weight": "embed"}),
        layers=layers,
        final_norm=norm("final.norm", role=""),
        head=PartSpec("head", {"vocab_size": cfg.vocab, "hidden_size": cfg.width, "tied": False,
                               "softcap": cfg.logit_softcap}, {"weight": "head"}),
    )


register_architecture("Lunerax", LuneraxConfig.from_dict, lunerax_plan, replace=True)
