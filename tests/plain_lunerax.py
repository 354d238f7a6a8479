"""A plain, slow implementation of the Lunerax design: whole sequences, no cache, float64, one function per mechanism.

It shares no code with the package.  ``cfg`` is the design's config.json as a dictionary and ``T`` maps checkpoint
names to tensors.  Notation: ``x`` the residual stream ``[n, width]``, ``h`` a sublayer's input.

* norm: ``L(x) = (x - mean) / sqrt(mean((x - mean)^2) + eps) * w + b``.
* layer: ``x += mixer(L1(x))``, then ``x += ff(L2(x))`` if it has a feed-forward, then the token's own input:
  ``x += rms(P (gelu(G x) * e)) * s`` with ``e`` the layer's part of a second embedding row of the token.
* mixers: the delta rule with a decay for every key channel, latent attention over a window, and grouped attention
  without positions whose scores are capped, whose window keeps the first tokens, and whose values are mixed with
  those of the first such layer.
* logits: ``c tanh(head L(x) / c)``.
"""

import math

import torch

F64 = torch.float64


def _t(T, name):
    return T[name].to(F64)


def lin(h, T, name):
    return h @ _t(T, name).T


def silu(z):
    return z * torch.sigmoid(z)


def rms(y, eps):
    return y / torch.sqrt((y * y).mean(-1, keepdim=True) + eps)


def layer_norm(x, T, name, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * _t(T, name) + _t(T, name + ".b")


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def soft_cap(z, cap):
    return z if cap is None else cap * torch.tanh(z / cap)


# ---------------------------------------------------------------------------------------------------------
# the delta rule with a decay per key channel
def causal_conv(u, w):
    """``out[t, c] = sum_j w[c, j] u[t - (taps - 1) + j, c]``: the last tap meets the current token, zeros stand
    before the sequence."""
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u])
    return sum(padded[j: j + u.shape[0]] * w[:, j] for j in range(taps))


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def channel_decay(h, T, p, heads, dim):
    """``[n, heads, dim]``: one factor in (0, 1) for every head and key channel."""
    z = lin(lin(h, T, p + ".a1"), T, p + ".a2") + _t(T, p + ".dt_bias")
    step = torch.nn.functional.softplus(z, threshold=1e9).reshape(-1, heads, dim)
    return torch.exp(-torch.exp(_t(T, p + ".A_log"))[:, None] * step)


def channel_delta_rule(q, k, v, beta, decay):
    """Per head: every row of the state fades by its own factor, what the key would read out now is replaced, in part,
    by the new value, and the query reads the state that already holds this token."""
    n, H, Dv = v.shape
    G, D = q.shape[1], q.shape[2]
    own = torch.arange(H) // (H // G)
    S = torch.zeros(H, D, Dv, dtype=F64)
    o = torch.zeros(n, H, Dv, dtype=F64)
    for t in range(n):
        kt, qt = k[t, own], q[t, own]
        S = decay[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - (S * kt[:, :, None]).sum(1))
        S = S + kt[:, :, None] * u[:, None, :]
        o[t] = (S * qt[:, :, None]).sum(1)
    return o


def channel_delta_mixer(h, T, p, mx, eps):
    n = h.shape[0]
    H, G, D, Dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    short = lambda name: silu(causal_conv(lin(h, T, f"{p}.{name}"), _t(T, f"{p}.{name}.conv")))
    q = unit(short("q").reshape(n, G, D)) * D ** -0.5
    k = unit(short("k").reshape(n, G, D))
    v = short("v").reshape(n, H, Dv)
    o = channel_delta_rule(q, k, v, torch.sigmoid(lin(h, T, p + ".b")), channel_decay(h, T, p, H, D))
    o = (rms(o, eps) * _t(T, p + ".norm")).reshape(n, H * Dv)
    return lin(o * torch.sigmoid(lin(lin(h, T, p + ".g1"), T, p + ".g2")), T, p + ".o")


# ---------------------------------------------------------------------------------------------------------
# attention
def rotate_half(x, rot):
    """``x [n, heads, dim]``: element ``i`` of the first ``dims`` turns with element ``i + dims / 2``."""
    dims = rot["dims"]
    f = rot["base"] ** (-2.0 * torch.arange(dims // 2, dtype=F64) / dims)
    a = torch.arange(x.shape[0], dtype=F64)[:, None] * f
    c, s = torch.cos(a)[:, None, :], torch.sin(a)[:, None, :]
    u, w = x[..., : dims // 2], x[..., dims // 2: dims]
    return torch.cat([u * c - w * s, w * c + u * s, x[..., dims:]], -1)


def visible(n, mask):
    """``[query, key]``: the last ``size`` positions, the query's own included, and the sequence's first ones; all of the
    past without a mask."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    if not mask:
        return j <= i
    return (j <= i) & ((i - j < mask["size"]) | (j < mask.get("keep_first", 0)))


def weights_over(scores, seen):
    return torch.softmax(scores.masked_fill(~seen, float("-inf")), -1)


def latent_attention(h, T, p, mx, eps):
    n = h.shape[0]
    H, D, R, Dv, r = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
    cq = rms(lin(h, T, p + ".dq"), eps) * _t(T, p + ".dq.norm")
    q = lin(cq, T, p + ".uq").reshape(n, H, D + R)
    down = lin(h, T, p + ".dkv")
    c = rms(down[:, :r], eps) * _t(T, p + ".dkv.norm")
    shared = rotate_half(down[:, None, r:], mx["rot"])[:, 0]
    qr = rotate_half(q[..., D:], mx["rot"])
    k = lin(c, T, p + ".uk").reshape(n, H, D)
    v = lin(c, T, p + ".uv").reshape(n, H, Dv)
    seen = visible(n, mx.get("mask"))
    out = torch.zeros(n, H, Dv, dtype=F64)
    for hd in range(H):
        out[:, hd] = weights_over((q[:, hd, :D] @ k[:, hd].T + qr[:, hd] @ shared.T) * mx["scale"], seen) @ v[:, hd]
    return lin(out.reshape(n, H * Dv) * torch.sigmoid(lin(h, T, p + ".g")), T, p + ".o")


def mixed_values(v, T, p, first):
    """The values of a layer that takes part in the mixing: its own, or a share of the first such layer's."""
    if first is None:
        return v
    lam = _t(T, p + ".vmix")
    return (1.0 - lam) * v + lam * first


def capped_attention(h, T, p, mx, first=None):
    """(result, the layer's values as they are cached); ``first``: the first mixing layer's values, if this layer
    mixes and is not that layer."""
    n = h.shape[0]
    H, G, D, Dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = lin(h, T, p + ".q").reshape(n, H, D)
    k = lin(h, T, p + ".k").reshape(n, G, D)
    v = mixed_values(lin(h, T, p + ".v").reshape(n, G, Dv), T, p, first)
    seen = visible(n, mx.get("mask"))
    out = torch.zeros(n, H, Dv, dtype=F64)
    for hd in range(H):
        g = hd // (H // G)
        out[:, hd] = weights_over(soft_cap((q[:, hd] @ k[:, g].T) * mx["scale"], mx.get("softcap")), seen) @ v[:, g]
    return lin(out.reshape(n, H * Dv) * torch.sigmoid(lin(h, T, p + ".g")), T, p + ".o"), v


# ---------------------------------------------------------------------------------------------------------
def gated_relu(h, T, p):
    return lin(torch.relu(lin(h, T, p + ".gate")) * lin(h, T, p + ".up"), T, p + ".down")


def token_input(x, T, p, rows, eps):
    """What a layer adds for the token itself; ``rows [n, dim]`` the layer's part of the tokens' second embedding."""
    y = lin(gelu_tanh(lin(x, T, p + ".side.gate")) * rows, T, p + ".side.proj")
    return rms(y, eps) * _t(T, p + ".side.norm")


def layer_streams(cfg, T, tokens):
    """The residual stream after every layer, ``[layers, n, width]``, and the last one normed."""
    eps = cfg["norm"]["eps"]
    ids = torch.as_tensor(tokens, dtype=torch.long)
    x = _t(T, "embed")[ids] * cfg["embedding"]["scale"]
    side = cfg["token_side"]["dim"] if cfg.get("token_side") else 0
    after, first = [], None
    for i, layer in enumerate(cfg["layers"]):
        p, mx = f"l{i}", layer["mixer"]
        h = layer_norm(x, T, p + ".norm1", eps)
        if layer["type"] == "channel_delta":
            y = channel_delta_mixer(h, T, p + ".mix", mx, eps)
        elif layer["type"] == "latent_attention":
            y = latent_attention(h, T, p + ".mix", mx, eps)
        elif layer["type"] == "attention":
            y, v = capped_attention(h, T, p + ".mix", mx, first if mx.get("v_mix") else None)
            if mx.get("v_mix") and first is None:
                first = v
        else:
            raise ValueError(layer["type"])
        x = x + y
        if layer.get("mlp") is not None:
            x = x + gated_relu(layer_norm(x, T, p + ".norm2", eps), T, p + ".mlp")
        if side:
            x = x + token_input(x, T, p, _t(T, "side.embed")[ids, i * side: (i + 1) * side], eps)
        after.append(x.clone())
    return torch.stack(after), layer_norm(x, T, "final.norm", eps)


def forward(cfg, T, tokens):
    """Logits ``[n, vocab]`` of a whole sequence."""
    return soft_cap(lin(layer_streams(cfg, T, tokens)[1], T, "head"), cfg.get("logit_softcap"))
