"""A plain, slow implementation of the Melerax design: whole sequences, no cache, float64, one function per mechanism.

It shares no code with the package.  ``cfg`` is the design's config.json as a dictionary and ``T`` maps checkpoint
names to tensors.  Notation: ``x`` the residual stream ``[n, width]``, which the sublayers read as it is.

* input: ``x = E[token] + B[row]``, the row chosen by the token and the one before it.
* layer: ``x += N1(mixer(x)) * s1``, then ``x += N2(ff(x)) * s2`` if it has a feed-forward; ``N(y) = rms(y) * (1 + w)``.
* mixers: grouped attention inside blocks of positions beside a gated linear recurrent unit (half the sum of their
  normed results), a matrix state with a decay per key channel and a bonus for the current token, and the recurrent
  unit alone.
* logits: ``head N(x)``.
"""

import math

import torch

F64 = torch.float64


def _t(T, name):
    return T[name].to(F64)


def lin(h, T, name, bias=False):
    y = h @ _t(T, name).T
    return y + _t(T, name + ".b") if bias else y


def rms(y, eps):
    return y / torch.sqrt((y * y).mean(-1, keepdim=True) + eps)


def offset_norm(y, w, eps):
    """The gain is stored as its distance from one."""
    return rms(y, eps) * (1.0 + w)


def silu(z):
    return z * torch.sigmoid(z)


def gelu_exact(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def causal_conv(u, w):
    """``out[t, c] = sum_j w[c, j] u[t - (taps - 1) + j, c]``: the last tap meets the current token, zeros stand
    before the sequence."""
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u])
    return sum(padded[j: j + u.shape[0]] * w[:, j] for j in range(taps))


# ---------------------------------------------------------------------------------------------------------
def pair_rows(tokens, bigram):
    """The row of the pair table for every token: the last row for a sequence's first token."""
    rows = []
    for i, tok in enumerate(tokens):
        rows.append(bigram["buckets"] if i == 0 else
                    (int(tokens[i - 1]) * bigram["mul_prev"] + int(tok) * bigram["mul_cur"]) % bigram["buckets"])
    return rows


def embed(cfg, T, tokens):
    x = _t(T, "embed")[torch.as_tensor(tokens, dtype=torch.long)]
    bigram = (cfg.get("embedding") or {}).get("bigram")
    return x if not bigram else x + _t(T, "bigram")[torch.as_tensor(pair_rows(tokens, bigram), dtype=torch.long)]


# ---------------------------------------------------------------------------------------------------------
# attention inside blocks of positions
def rotate_pairs(x, rot):
    """``x [n, heads, dim]``: elements ``2i`` and ``2i + 1`` of the first ``dims`` turn together."""
    n, heads, _ = x.shape
    dims = rot["dims"]
    f = rot["base"] ** (-2.0 * torch.arange(dims // 2, dtype=F64) / dims)
    a = torch.arange(n, dtype=F64)[:, None] * f
    c, s = torch.cos(a)[:, None, :], torch.sin(a)[:, None, :]
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    turned = torch.stack([u * c - v * s, v * c + u * s], -1).reshape(n, heads, dims)
    return torch.cat([turned, x[..., dims:]], -1)


def visible(n, mask):
    """``[query, key]``: the past inside the query's own block of positions, all of it without a mask."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    seen = j <= i
    return seen if not mask else seen & (i // mask["size"] == j // mask["size"])


def soft_cap(z, cap):
    return z if cap is None else cap * torch.tanh(z / cap)


def block_attention(h, T, p, mx, eps):
    n = h.shape[0]
    H, G, D, Dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    short = lambda name: causal_conv(lin(h, T, f"{p}.{name}", bias=True), _t(T, f"{p}.{name}.conv"))
    q = (rms(short("q"), eps) * _t(T, p + ".q.norm")).reshape(n, H, D)
    k = (rms(short("k"), eps) * _t(T, p + ".k.norm")).reshape(n, G, D)
    v = short("v").reshape(n, G, Dv)
    if mx.get("rot"):
        q, k = rotate_pairs(q, mx["rot"]), rotate_pairs(k, mx["rot"])
    seen = visible(n, mx.get("mask"))
    out = torch.zeros(n, H, Dv, dtype=F64)
    for hd in range(H):
        g = hd // (H // G)
        scores = soft_cap((q[:, hd] @ k[:, g].T) * mx["scale"], mx.get("softcap"))
        out[:, hd] = torch.softmax(scores.masked_fill(~seen, float("-inf")), -1) @ v[:, g]
    return lin(out.reshape(n, H * Dv), T, p + ".o")


# ---------------------------------------------------------------------------------------------------------
# the gated linear recurrent unit
def block_gate(u, w, b):
    """A sigmoid gate from equal parts of ``u``, each through a square matrix of its own."""
    blocks, size = b.shape
    parts = u.reshape(-1, blocks, size)
    return torch.sigmoid(torch.stack([parts[:, i] @ w[i].T + b[i] for i in range(blocks)], 1)).reshape(u.shape)


def linear_unit(u, r, i, lam):
    """``S <- a S + sqrt(1 - a^2) i u`` with ``a = exp(-8 r softplus(lam))``, from zero."""
    a = torch.exp(-8.0 * r * torch.nn.functional.softplus(lam, threshold=1e9))
    S, out = torch.zeros(u.shape[1], dtype=F64), torch.zeros_like(u)
    for t in range(u.shape[0]):
        S = a[t] * S + torch.sqrt(1.0 - a[t] * a[t]) * i[t] * u[t]
        out[t] = S
    return out


def recurrent_block(h, T, p):
    y = gelu_tanh(lin(h, T, p + ".y", bias=True))
    u = causal_conv(lin(h, T, p + ".x", bias=True), _t(T, p + ".conv")) + _t(T, p + ".conv.b")
    r = block_gate(u, _t(T, p + ".ra"), _t(T, p + ".ra.b"))
    i = block_gate(u, _t(T, p + ".ri"), _t(T, p + ".ri.b"))
    return lin(linear_unit(u, r, i, _t(T, p + ".lam")) * y, T, p + ".o")


def side_by_side(h, T, p, mx, eps):
    left = rms(block_attention(h, T, p + ".left", mx["left"], eps), eps) * _t(T, p + ".left.out")
    right = rms(recurrent_block(h, T, p + ".right"), eps) * _t(T, p + ".right.out")
    return 0.5 * (left + right)


# ---------------------------------------------------------------------------------------------------------
# the matrix state with a bonus
def token_shift(h, mu):
    before = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    return h + (before - h) * mu


def bonus_recurrence(r, k, v, w, u):
    """Per head: the query reads the state before this token plus the token's own write scaled by ``u``; then the rows
    of the state fade by ``w`` and the write is added."""
    n, H, D = k.shape
    S = torch.zeros(H, D, v.shape[2], dtype=F64)
    o = torch.zeros_like(v)
    for t in range(n):
        write = k[t][:, :, None] * v[t][:, None, :]
        o[t] = ((S + u[:, :, None] * write) * r[t][:, :, None]).sum(1)
        S = w[t][:, :, None] * S + write
    return o


def wkv_mixer(h, T, p, mx, eps):
    n, H, D = h.shape[0], mx["heads"], mx["dim"]
    mix = {s: token_shift(h, _t(T, f"{p}.mu.{s}")) for s in "rkvgw"}
    r, k, v = (lin(mix[s], T, f"{p}.{s}").reshape(n, H, D) for s in "rkv")
    z = lin(torch.tanh(lin(mix["w"], T, p + ".w1")), T, p + ".w2") + _t(T, p + ".w0")
    w = torch.exp(-torch.exp(z)).reshape(n, H, D)
    o = rms(bonus_recurrence(r, k, v, w, _t(T, p + ".u")), eps).reshape(n, H * D)
    return lin(o * _t(T, p + ".norm") * silu(lin(mix["g"], T, p + ".g")), T, p + ".o")


# ---------------------------------------------------------------------------------------------------------
def gated_dense(h, T, p):
    return lin(gelu_tanh(lin(h, T, p + ".gate", bias=True)) * lin(h, T, p + ".up", bias=True), T, p + ".down", bias=True)


def expert(h, T, p):
    return lin(gelu_exact(lin(h, T, p + ".up")), T, p + ".down")


def routing(h, T, p, top):
    """``[n, experts]``: a token's weights, zero for the experts it does not take."""
    z = lin(h, T, p + ".router", bias=True)
    best = z.topk(top, -1)
    return torch.zeros_like(z).scatter(-1, best.indices, torch.softmax(best.values, -1))


def routed_experts(h, T, p, mlp):
    weights = routing(h, T, p, mlp["router"]["top"])
    y = sum(weights[:, e: e + 1] * expert(h, T, f"{p}.e{e}") for e in range(mlp["router"]["experts"]))
    return y + expert(h, T, p + ".shared") if mlp.get("shared") else y


def layer_streams(cfg, T, tokens):
    """The residual stream after every layer, ``[layers, n, width]``, and the last one normed."""
    eps = cfg["norm"]["eps"]
    x = embed(cfg, T, tokens)
    after = []
    for i, layer in enumerate(cfg["layers"]):
        p, mx = f"l{i}", layer["mixer"]
        if layer["type"] == "parallel":
            y = side_by_side(x, T, p + ".mix", mx, eps)
        elif layer["type"] == "wkv":
            y = wkv_mixer(x, T, p + ".mix", mx, eps)
        elif layer["type"] == "rglru":
            y = recurrent_block(x, T, p + ".mix")
        else:
            raise ValueError(layer["type"])
        x = x + offset_norm(y, _t(T, p + ".norm1"), eps) * _t(T, p + ".ls1")
        mlp = layer.get("mlp")
        if mlp is not None:
            y = gated_dense(x, T, p + ".mlp") if mlp["kind"] == "dense" else routed_experts(x, T, p + ".mlp", mlp)
            x = x + offset_norm(y, _t(T, p + ".norm2"), eps) * _t(T, p + ".ls2")
        after.append(x.clone())
    return torch.stack(after), offset_norm(x, _t(T, "final.norm"), eps)


def forward(cfg, T, tokens):
    """Logits ``[n, vocab]`` of a whole sequence."""
    return lin(layer_streams(cfg, T, tokens)[1], T, "head")
