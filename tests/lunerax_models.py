"""Small Lunerax configurations for the tests, their model folders, and runners over them.

The configurations differ from one another in every size and option: delta rules with as many query/key heads as value
heads and with fewer, key and value widths that differ, convolutions of 1 to 5 taps, low-rank pairs of every rank;
latent attention with windows shorter and longer than a page and without one, rotations of all of the rotated part and
of some of it; capped attention with one key/value head and several, with and without a cap, a window, kept first tokens
(fewer and more than a page holds, more than the window), with and without mixed values; layers without a feed-forward;
every order of the three mixers; with and without a second embedding and a cap on the logits.
"""

from __future__ import annotations

import copy
import json

import torch
from safetensors import safe_open

import plain_lunerax as plain
from mogisun_models import TOLERANCE, err, make_runner, rel_err, rms_err  # noqa: F401  (the same runners and measures)


def delta(heads, kv_heads, dim, vdim, conv, decay_rank, gate_rank):
    return {"type": "channel_delta", "mixer": {"conv": conv, "dim": dim, "heads": heads, "kv_heads": kv_heads, "vdim": vdim,
                                               "decay_rank": decay_rank, "gate_rank": gate_rank}}


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, window, scale, base, dims=None):
    mixer = {"dim": dim, "heads": heads, "kv_rank": kv_rank, "q_rank": q_rank, "rot": {"base": base, "dims": dims or rot_dim},
             "rot_dim": rot_dim, "scale": scale, "vdim": vdim}
    if window:
        mixer["mask"] = {"size": window}
    return {"type": "latent_attention", "mixer": mixer}


def attention(heads, kv_heads, dim, vdim, window, keep, scale, cap, v_mix):
    mixer = {"dim": dim, "heads": heads, "kv_heads": kv_heads, "scale": scale, "v_mix": v_mix, "vdim": vdim}
    if cap:
        mixer["softcap"] = cap
    if window:
        mixer["mask"] = {"keep_first": keep, "size": window}
    return {"type": "attention", "mixer": mixer}


def layer(mixer, ff):
    return dict(mixer, mlp={"kind": "dense", "ff": ff} if ff else None)


def model(vocab, width, eps, scale, side, cap, layers):
    cfg = {"architecture": "Lunerax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
           "layers": layers}
    if side:
        cfg["token_side"] = {"dim": side}
    if cap:
        cfg["logit_softcap"] = cap
    return cfg


CONFIGS = {
    # the three mixers in turn; windows shorter than two pages; kept tokens that fill more than a page; value widths of
    # their own; the mixing layers share their value heads, an attention layer between them does not mix
    "a": model(211, 96, 1e-5, 4.0, 20, 12.0, [
        layer(attention(4, 2, 24, 16, 11, 3, 0.3, 5.0, True), 72),
        layer(delta(4, 2, 12, 20, 4, 10, 14), 40),
        layer(latent(3, 16, 8, 24, 20, 40, 13, 0.25, 10000.0), 72),
        layer(attention(3, 1, 16, 40, 9, 12, 0.4, None, False), None),
        layer(delta(3, 3, 16, 8, 2, 24, 6), None),
        layer(attention(2, 2, 32, 16, 30, 0, 0.2, 2.0, True), 56)]),
    # one head everywhere; a convolution of one tap (no inputs to keep); a window of one token; one kept token; no cap
    "b": model(160, 64, 3e-6, 1.0, 1, None, [
        layer(delta(1, 1, 32, 32, 1, 1, 1), 48),
        layer(attention(1, 1, 32, 32, 1, 1, 0.25, 30.0, True), 40),
        layer(latent(1, 24, 2, 40, 16, 24, 1, 0.3, 1000.0), None),
        layer(attention(1, 1, 32, 32, 50, 40, 1.0, 1.0, True), 64)]),
    # sizes at which the GPU takes its matrix-core attention and its few-row products
    "c": model(300, 128, 1e-6, 8.0, 64, 20.0, [
        layer(delta(4, 2, 64, 32, 3, 32, 16), 256),
        layer(attention(8, 2, 64, 64, 40, 5, 0.125, 8.0, True), 192),
        layer(latent(4, 32, 32, 64, 64, 96, 50, 0.12, 50000.0), 256),
        layer(delta(2, 2, 32, 64, 4, 64, 64), None),
        layer(attention(4, 2, 128, 64, 70, 20, 0.09, 15.0, True), 128),
        layer(latent(6, 16, 16, 32, 64, 112, 24, 0.2, 500.0, dims=8), 128)]),
    # sizes that are multiples of nothing the kernels like: every vector path has to step aside; no windows on some
    "e": model(131, 100, 2e-6, 1.3, 7, 3.0, [
        layer(latent(5, 12, 6, 20, 14, 22, None, 0.4, 777.0, dims=4), 52),
        layer(attention(6, 3, 12, 10, 17, 19, 0.3, 4.0, False), 36),
        layer(delta(6, 2, 10, 14, 5, 9, 11), 44),
        layer(attention(5, 5, 20, 12, None, 0, 0.25, 6.0, True), None),
        layer(attention(5, 5, 12, 12, 23, 2, 0.4, 50.0, True), 30)]),
    # no second embedding, a latent wider than any head the matrix-core attention is built for, heads of 144
    "f": model(97, 72, 1e-4, 2.5, None, 7.0, [
        layer(latent(2, 32, 32, 40, 24, 288, 33, 0.1, 10000.0), 64),
        layer(attention(2, 1, 144, 144, 21, 9, 0.08, 10.0, True), 40),
        layer(delta(2, 1, 24, 40, 2, 8, 8), 40)]),
}

PAGE_SIZE = {"a": 8, "b": 16, "c": 16, "e": 16, "f": 8}


def tame(tensors, seed=0):
    """Vectors that the random mode draws around 1 and that mean something else: biases and decay rates around 0, shares
    of the value mixing between 0 and 1, convolution weights of a size that keeps the recurrences lively."""
    g = torch.Generator().manual_seed(1000 + seed)
    for name, t in tensors.items():
        draw = lambda std: torch.randn(t.shape, generator=g) * std
        if name.endswith((".b", ".dt_bias", ".A_log")) and t.dim() == 1:
            t.copy_(draw(0.4))
        elif name.endswith(".conv"):
            t.copy_(draw(0.5))
        elif name.endswith(".vmix"):
            t.copy_(0.2 + 0.7 * torch.rand(t.shape, generator=g))


def write_model(folder, name_or_config, seed=0, std=0.08, spread=0.3, change=None):
    """config.json + model.safetensors with the package's random mode: matrices N(0, std), vectors 1 + N(0, spread),
    then ``tame``; ``change(tensors)`` may edit the tensors before they are written.  The written config.json does not
    name the ranks of the low-rank pairs (the loader reads them from the tensors)."""
    from simple_inference_amd.config import EngineConfig
    from simple_inference_amd.engine import build_model
    from simple_inference_amd.weights import random_tensors, write_model_folder

    cfg = copy.deepcopy(CONFIGS[name_or_config] if isinstance(name_or_config, str) else name_or_config)
    built, mcfg = build_model(cfg, EngineConfig(device="cpu", dtype="float32", max_seq_len=64), kernels=None)
    tensors = random_tensors(built.expected_tensors(), seed, std, spread, "bfloat16")
    tame(tensors, seed)
    if change is not None:
        change(tensors)
    out = mcfg.to_dict()
    for entry in out["layers"]:
        for key in ("decay_rank", "gate_rank"):
            entry["mixer"].pop(key, None)
    write_model_folder(folder, out, tensors)
    return folder


def read_model(folder):
    with open(f"{folder}/config.json") as f:
        cfg = json.load(f)
    w = {}
    with safe_open(f"{folder}/model.safetensors", framework="pt") as f:
        for k in f.keys():
            w[k] = f.get_tensor(k).double()
    return cfg, w


def plain_logits(folder, tokens):
    cfg, w = read_model(folder)
    return plain.forward(cfg, w, tokens).float()
