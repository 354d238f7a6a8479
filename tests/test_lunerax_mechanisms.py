"""Every mechanism of the Lunerax design alone: the kernel (its torch twin on the CPU, the HIP kernel on the GPU in
float32 and bfloat16) against the plain implementation's function for it, at sizes of all kinds."""

import types

import pytest
import torch

import plain_lunerax as plain
from simple_inference_amd.cache import CacheManager
from simple_inference_amd.parts import FEED_FORWARDS, MIXERS, NORMS, TOKEN_INPUTS, BuildEnv, PagedKVNeed
from simple_inference_amd.parts.context import LayerCache, ResidualStream
from simple_inference_amd.parts.model import CacheLayout
from test_famepel_mechanisms import done, f32, portions, rounded, rows_of
from test_feduzen_mechanisms import empty_cache, fill_cache_by_pages, step_context
from test_mogisun_mechanisms import BACKENDS, close, context, lowered, rnd, setup


def env_for(k, dev, dtype):
    return BuildEnv(kernels=k, device=torch.device(dev), dtype=dtype, max_positions=2048)


def bind_part(part, g, dev, dtype, names, std=0.3, **fixed):
    """Random tensors for a part, bound to it; returns the same numbers in float64 under the plain names.  A vector named
    ``*norm`` or ``weight`` is drawn around one; ``fixed`` gives a tensor's size where the part leaves it open (a list)
    or its values."""
    bound, T = {}, {}
    for name, spec in part.weight_specs().items():
        given = fixed.get(name)
        shape = given if isinstance(given, (list, tuple)) else spec.shape
        t = given.double() if isinstance(given, torch.Tensor) else rnd(g, *shape, std=std) + (1.0 if name.endswith(("norm", "weight")) and spec.role == "vector" else 0.0)
        bound[name], T[names.get(name, "m." + name)] = lowered(t, torch.float32 if spec.role in ("vector", "float_matrix") else dtype, dev)
    part.bind(bound)
    return T


# ---------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width", [96, 50, 176, 1024, 2056, 8200])
def test_layer_norm_of_the_sum_and_of_the_normed_sum(backend, width):
    """``x += d`` or ``x += rms(d) s``, and the layer norm of the sum: all rows (the residual keeps the sum), chosen rows
    (it does not), nothing pending; the rows' mean is large against their spread.  And the sum alone, lowered."""
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(width)
    n, eps, post_eps = 7, 1e-5, 3e-4
    res = rnd(g, n, width, std=2.0) + 5.0
    d, d64 = lowered(rnd(g, n, width, std=1.5), dtype, dev)
    gain, w, b = 1 + rnd(g, width, std=0.3), 1 + rnd(g, width, std=0.3), rnd(g, width, std=0.4)
    T = {"w": rounded(w), "w.b": rounded(b)}
    args = (f32(w, dev), f32(b, dev), eps, dtype)
    rows = torch.tensor([5, 0, 5], dtype=torch.int32, device=dev)
    for post, added in ((None, d64), ((f32(gain, dev), post_eps), plain.rms(d64, post_eps) * rounded(gain))):
        want_sum = rounded(res) + added
        want = plain.layer_norm(want_sum, T, "w", eps)
        r = f32(res, dev)
        out = k.add_layernorm(r, d, post, *args)
        close(r, want_sum, 3e-6)
        close(out, want, tol)
        r = f32(res, dev)
        out = k.add_layernorm(r, d, post, *args, rows)
        close(r, rounded(res), 0)
        close(out, want[[5, 0, 5]], tol)
    r = f32(res, dev)
    close(k.add_layernorm(r, None, None, *args), plain.layer_norm(rounded(res), T, "w", eps), tol)
    r = f32(res, dev)
    low = k.add_lowered(r, d, dtype)
    close(r, rounded(res) + d64, 3e-6)
    assert low.dtype == dtype and torch.equal(low.float(), r.to(dtype).float())


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width,dim,first", [(64, 24, 5), (128, 64, 0), (96, 1, 3), (50, 19, 40), (256, 130, 64)])
@pytest.mark.parametrize("n", [1, 5, 40])
def test_what_a_layer_takes_of_the_token_itself(backend, width, dim, first, n):
    """The part with its norm, as the block arranges them, behind a result that is still pending."""
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(width + n)
    vocab, table_width, eps = 37, first + dim + 3, 1e-5
    env = env_for(k, dev, dtype)
    part = TOKEN_INPUTS.get("gated_embedding")({"hidden_size": width, "vocab_size": vocab, "dim": dim, "first_column": first,
                                                "table_width": table_width, "activation": "gelu_tanh"}, env)
    norm = NORMS.get("rmsnorm")({"size": width, "eps": eps}, env)
    T = bind_part(part, g, dev, dtype, {"gate": "l.side.gate", "proj": "l.side.proj", "table": "table"})
    T.update(bind_part(norm, g, dev, dtype, {"weight": "l.side.norm"}))
    ids = torch.randint(0, vocab, (n,), generator=g, dtype=torch.int32)
    res = rnd(g, n, width)
    d, d64 = lowered(rnd(g, n, width), dtype, dev)
    stream = ResidualStream(f32(res, dev))
    stream.delta = d
    x = stream.lower(k, dtype)
    assert stream.raw_delta is None
    x64 = x.double().cpu().clone()          # in float32 the rows are the residual itself, which grows below
    want = rounded(res) + d64
    close(stream.residual, want, 3e-6)
    stream.delta = part.forward(x, types.SimpleNamespace(token_ids=ids.to(dev)))
    stream.post = norm
    after = NORMS.get("layernorm")({"size": width, "eps": eps}, env)
    T.update(bind_part(after, g, dev, dtype, {"weight": "n", "bias": "n.b"}))
    out = after.forward(stream)
    rows = T["table"][ids.long(), first:first + dim]
    want = want + plain.token_input(x64, T, "l", rows, eps)
    close(stream.residual, want, tol)
    close(out, plain.layer_norm(want, T, "n", eps), tol)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("n,width,inter", [(5, 64, 40), (33, 128, 72), (19, 50, 27), (1, 192, 96)])
def test_the_rectified_gate(backend, n, width, inter):
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(n)
    part = FEED_FORWARDS.get("swiglu")({"hidden_size": width, "intermediate_size": inter, "activation": "relu"}, env_for(k, dev, dtype))
    T = bind_part(part, g, dev, dtype, {}, std=0.2)
    h, h64 = lowered(rnd(g, n, width), dtype, dev)
    close(done(part.forward(h, None)), plain.gated_relu(h64, T, "m"), tol * 2)
    assert part.plain_form() is None       # a kernel that runs whole blocks with the silu gate must leave this one alone


# ---------------------------------------------------------------------------------------------------------------
DELTA_SHAPES = [(4, 2, 12, 20, 10, 7), (1, 1, 8, 8, 1, 1), (2, 2, 64, 64, 32, 64), (4, 1, 128, 128, 128, 24), (6, 3, 56, 24, 40, 8),
                (1, 1, 40, 200, 16, 72), (2, 1, 264, 96, 33, 9)]


def channel_reference(qkv64, proj64, cols, T, H, G, D, Dv, eps):
    """The plain functions on convolved rows."""
    n = qkv64.shape[0]
    q = plain.unit(qkv64[:, :G * D].reshape(n, G, D)) * D ** -0.5
    kk = plain.unit(qkv64[:, G * D:2 * G * D].reshape(n, G, D))
    v = qkv64[:, 2 * G * D:].reshape(n, H, Dv)
    z = proj64[:, cols[1]:cols[1] + T["a2"].shape[1]] @ T["a2"].T + T["dt_bias"]
    step = torch.nn.functional.softplus(z, threshold=1e9).reshape(n, H, D)
    decay = torch.exp(-torch.exp(T["A_log"])[:, None] * step)
    o = plain.rms(plain.channel_delta_rule(q, kk, v, torch.sigmoid(proj64[:, cols[0]:cols[0] + H]), decay), eps) * T["norm"]
    return o.reshape(n, H * Dv) * torch.sigmoid(proj64[:, cols[2]:cols[2] + T["g2"].shape[1]] @ T["g2"].T)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("H,G,D,Dv,ra,rg", DELTA_SHAPES)
def test_the_rule_with_a_decay_per_channel_carries_its_state_through_any_cut(backend, H, G, D, Dv, ra, rg):
    """Three sequences of unequal length in scattered slots, fed in portions of unequal sizes down to one token, the
    batch's order changing: every output is the plain recurrence's over the whole sequence, and nobody else's slot is
    touched.  The matrices lie at the front of a longer state row; the low-rank columns lie aligned or not."""
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(H * 1000 + D)
    lengths, slots = [38, 6, 22], [4, 0, 2]
    start = 8 if ra % 8 == 0 else 3
    cols = (0, start + H + (-(start + H)) % start, 0)
    cols = (cols[0], cols[1], cols[1] + ra + (-ra) % 8)
    width = cols[2] + rg + (-rg) % 8
    width += (-width) % 8 if ra % 8 == 0 else 1
    qkvs = [lowered(rnd(g, n, 2 * G * D + H * Dv), dtype, dev) for n in lengths]
    projs = [lowered(rnd(g, n, width, std=1.0), dtype, dev) for n in lengths]
    a2, a2_64 = lowered(rnd(g, H * D, ra, std=ra ** -0.5), dtype, dev)
    g2, g2_64 = lowered(rnd(g, H * Dv, rg, std=rg ** -0.5), dtype, dev)
    T = {"A_log": rounded(rnd(g, H, std=0.7)), "dt_bias": rounded(rnd(g, H * D, std=0.7)), "norm": rounded(1 + rnd(g, Dv, std=0.3)),
         "a2": a2_64, "g2": g2_64}
    tail = 5
    state = torch.zeros(6, H * D * Dv + tail, dtype=torch.float32, device=dev)
    state[:, H * D * Dv:] = 3.0
    eps = 1e-5
    offsets = [sum(lengths[:s]) for s in range(len(lengths))]
    got = torch.zeros(sum(lengths), H * Dv, dtype=torch.float64)
    for step in portions(lengths, [2, 1, 9, 1, 3, 17]):
        ctx = context(dev, [n for _, _, n in step], [slots[s] for s, _, _ in step])
        pick = lambda rows: torch.cat([rows[s][0][a:a + n] for s, a, n in step]).contiguous()
        out = k.channel_delta_rule(pick(qkvs), pick(projs), cols, a2, g2, f32(T["A_log"], dev), f32(T["dt_bias"], dev),
                                   f32(T["norm"], dev), H, G, D, Dv, eps, ctx, state)
        got[rows_of(step, offsets)] = out.double().cpu()
    want = torch.cat([channel_reference(qkvs[s][1], projs[s][1], cols, T, H, G, D, Dv, eps) for s in range(len(lengths))])
    close(got, want, tol * 2)
    assert float(state[[1, 3, 5], :H * D * Dv].abs().max()) == 0.0
    assert float((state[:, H * D * Dv:] - 3.0).abs().max()) == 0.0      # what lies behind the matrices is not theirs


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("n,rank", [(1, 16), (16, 128), (64, 8), (65, 40), (200, 72), (70, 13)])
def test_low_rank_pairs_of_many_and_few_tokens(backend, n, rank):
    """One token at a time nothing is remembered (a fresh slot each): what a token's output owes to the decays is nothing,
    so the steps of many tokens are read through the recurrence of ``n`` tokens; every token's decays and gates differ."""
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(n * 100 + rank)
    H, G, D, Dv = 3, 3, 24, 40
    cols = (0, 8, 8 + rank + (-rank) % 8)
    width = cols[2] + rank + (-rank) % 8
    qkv, qkv64 = lowered(rnd(g, n, 2 * G * D + H * Dv), dtype, dev)
    proj, proj64 = lowered(rnd(g, n, width), dtype, dev)
    a2, a2_64 = lowered(rnd(g, H * D, rank, std=2 * rank ** -0.5), dtype, dev)
    g2, g2_64 = lowered(rnd(g, H * Dv, rank, std=2 * rank ** -0.5), dtype, dev)
    T = {"A_log": rounded(rnd(g, H, std=0.5) - 1.0), "dt_bias": rounded(rnd(g, H * D) - 1.0), "norm": torch.ones(Dv, dtype=torch.float64),
         "a2": a2_64, "g2": g2_64}
    state = torch.zeros(1, H * D * Dv, dtype=torch.float32, device=dev)
    out = k.channel_delta_rule(qkv, proj, cols, a2, g2, f32(T["A_log"], dev), f32(T["dt_bias"], dev), f32(T["norm"], dev), H, G, D, Dv,
                               1e-5, context(dev, [n], [0]), state)
    close(out, channel_reference(qkv64, proj64, cols, T, H, G, D, Dv, 1e-5), tol * 2)


@pytest.mark.parametrize("backend", BACKENDS)
def test_every_key_channel_forgets_at_its_own_rate_and_a_second_write_replaces_the_first(backend):
    """Built inputs: two key channels are written once each with values of their own; one channel's decay keeps nearly
    all of it over 300 tokens, the other's nothing.  A query along both then reads the first value only (one decay for
    the whole head would keep or lose both).  A second write along the slow channel at full strength replaces what it
    held."""
    k, dev, dtype, tol = setup(backend)
    H = G = 1
    D, Dv, n = 16, 8, 330
    g = torch.Generator().manual_seed(1)
    cols = (0, 8, 16)
    e = torch.eye(D, dtype=torch.float64)
    qkv = torch.zeros(n, 2 * D + Dv, dtype=torch.float64)
    proj = torch.zeros(n, 24, dtype=torch.float64)
    proj[:, 0] = 30.0                                 # write at full strength
    proj[:, 8] = proj[:, 16] = 1.0
    for t in range(n):
        qkv[t, D:2 * D] = e[2 + t % (D - 2)]
        qkv[t, :D] = e[0] + e[1]                      # everybody asks along the first two channels
        qkv[t, 2 * D:] = rnd(g, Dv)
    a, b, c = torch.arange(Dv, dtype=torch.float64) - 3.5, torch.linspace(2, -1, Dv, dtype=torch.float64), torch.ones(Dv, dtype=torch.float64)
    qkv[5, D:2 * D], qkv[5, 2 * D:] = e[0], a
    qkv[6, D:2 * D], qkv[6, 2 * D:] = e[1], b
    again = qkv.clone()
    again[310, D:2 * D], again[310, 2 * D:] = e[0], c
    a2 = torch.zeros(D, 8, dtype=torch.float64)
    a2[:, 0] = -8.0                                   # small steps: slow decay
    a2[1, 0] = 1.0                                    # but for the second channel
    g2 = torch.zeros(Dv, 8, dtype=torch.float64)
    g2[:, 0] = 4.0                                    # an open output gate
    w, w64 = lowered(a2, dtype, dev)
    o, o64 = lowered(g2, dtype, dev)
    T = {"A_log": torch.zeros(1, dtype=torch.float64), "dt_bias": torch.zeros(D, dtype=torch.float64),
         "norm": torch.ones(Dv, dtype=torch.float64), "a2": w64, "g2": o64}
    outs = {}
    for name, rows in (("once", qkv), ("again", again)):
        state = torch.zeros(2, D * Dv, dtype=torch.float32, device=dev)
        x, x64 = lowered(rows, dtype, dev)
        p, p64 = lowered(proj, dtype, dev)
        got = []
        for lo, hi in [(0, 7), (7, 9)] + [(t, t + 1) for t in range(9, n)]:      # a portion, two tokens, then decoding
            got.append(k.channel_delta_rule(x[lo:hi].contiguous(), p[lo:hi].contiguous(), cols, w, o, f32(T["A_log"], dev),
                                            f32(T["dt_bias"], dev), f32(T["norm"], dev), H, G, D, Dv, 1e-6,
                                            context(dev, [hi - lo], [1]), state))
        outs[name] = torch.cat(got).double().cpu()
        close(outs[name], channel_reference(x64, p64, cols, T, H, G, D, Dv, 1e-6), tol * 2)
    cos = lambda u, v: float((u * v).sum() / u.norm() / v.norm())
    assert cos(outs["once"][6], a) < 0.99                       # both values are there at first
    assert cos(outs["once"][n - 1], a) > 0.99 and cos(outs["again"][309], a) > 0.99
    assert cos(outs["again"][n - 1], c) > 0.99


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("mx,ranks", [(dict(heads=4, kv_heads=2, dim=12, vdim=20, conv=4), (10, 14)),
                                      (dict(heads=2, kv_heads=2, dim=64, vdim=32, conv=3), (24, 24)),
                                      (dict(heads=1, kv_heads=1, dim=32, vdim=48, conv=1), (1, 5))])
def test_the_channel_delta_part_is_the_plain_mixer(backend, mx, ranks):
    """The part as the plan builds it (stacked projections with every part aligned, ranks read from the tensors)."""
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(11)
    hidden, n, H, G = 64, 31, mx["heads"], mx["kv_heads"]
    part = MIXERS.get("channel_delta")({"hidden_size": hidden, "num_heads": H, "num_kv_heads": G, "key_dim": mx["dim"],
                                        "value_dim": mx["vdim"], "conv_taps": mx["conv"], "norm_eps": 1e-5}, env_for(k, dev, dtype))
    names = {"q_conv": "m.q.conv", "k_conv": "m.k.conv", "v_conv": "m.v.conv", "a_log": "m.A_log"}
    T = bind_part(part, g, dev, dtype, names, std=0.2, a1=[ranks[0], hidden], a2=[H * mx["dim"], ranks[0]], g1=[ranks[1], hidden],
                  g2=[H * mx["vdim"], ranks[1]], norm=1 + rnd(g, mx["vdim"], std=0.2))
    h, h64 = lowered(rnd(g, n, hidden), dtype, dev)
    state = torch.zeros(2, *part.state_need().shape, dtype=torch.float32, device=dev)
    outs = []
    for lo, hi in ((0, 17), (17, 19), (19, 20), (20, 21), (21, n)):
        outs.append(done(part.forward(h[lo:hi].contiguous(), context(dev, [hi - lo], [1]), LayerCache(state=state))))
    close(torch.cat(outs), plain.channel_delta_mixer(h64, T, "m", mx, 1e-5), tol * 3)
    with pytest.raises(ValueError):
        bind_part(part, g, dev, dtype, names, a1=[7, hidden], a2=[H * mx["dim"], 6], g1=[5, hidden], g2=[H * mx["vdim"], 5])


# ---------------------------------------------------------------------------------------------------------------
def plain_scores(q, keys, values, qpos, scale, cap, mask):
    """q [n, H, dim] at positions ``qpos`` over keys and values [T, G, .] of one sequence, by the plain functions."""
    H, G, T = q.shape[1], keys.shape[1], keys.shape[0]
    seen = plain.visible(T, mask)[qpos]
    out = []
    for h in range(H):
        kk, v = keys[:, h // (H // G)].double(), values[:, h // (H // G)].double()
        out.append(plain.weights_over(plain.soft_cap((q[:, h].double() @ kk.T) * scale, cap), seen) @ v)
    return torch.stack(out, 1)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("heads,kv,dim,window,keep,cap,page", [
    (3, 3, 32, 24, 3, 2.0, 8), (4, 2, 16, 20, 20, None, 16), (8, 2, 64, 37, 70, 1.5, 16), (6, 1, 32, None, 0, 3.0, 8),
    (4, 4, 128, 64, 1, 4.0, 16), (2, 1, 144, 33, 9, 2.0, 32), (2, 2, 256, 41, 65, 2.5, 16), (6, 3, 80, 61, 6, 10.0, 64),
    (20, 1, 32, 50, 7, 2.0, 16), (2, 2, 24, 18, 6, 2.0, 4)])
def test_capped_scores_and_kept_first_positions_in_prompts_and_decoding(backend, heads, kv, dim, window, keep, cap, page):
    """A whole prompt, portions that begin inside and behind the kept positions, single tokens around the window's and
    the kept positions' edges.  Pages that nobody may look at (between the kept positions and a window) have no entry in
    the block table."""
    k, dev, dtype, tol = setup(backend)
    scale, T = 0.31, 400
    mask = {"size": window, "keep_first": keep} if window else None
    w = window or 32
    runs = [(0, T), (keep + w + 3, 2 * w), (300, 60), (w, 1), (w + keep, 1), (w + keep - 1 if w + keep else 0, 1), (3 * page, 1), (0, 1),
            (399, 1), (200, 2)]
    ctx, table, n_pages, runs = step_context(dev, runs, page, k)
    cache = empty_cache(dev, dtype, n_pages, kv, page, dim, dim, table)
    qkv = torch.zeros(ctx.n_tokens, heads * dim + 2 * kv * dim, dtype=dtype)
    g = torch.Generator().manual_seed(dim)
    want, row = [], 0
    for s, (first, n) in enumerate(runs):
        L = first + n
        keys, values = rnd(g, L, kv, dim).to(dtype), rnd(g, L, kv, dim).to(dtype)
        q = rnd(g, n, heads, dim).to(dtype)
        fill_cache_by_pages(cache, table.cpu(), keys, values, page, s)
        qkv[row:row + n, :heads * dim] = q.reshape(n, heads * dim)
        want.append(plain_scores(q, keys, values, list(range(first, L)), scale, cap, mask))
        row += n
    if window:
        held = table.clone()
        for s, (first, n) in enumerate(runs):
            for i in range(-(-keep // page), max(0, first - window + 1) // page):
                held[s, i] = -1
        cache.block_table = held
    got = k.paged_attention(qkv.to(dev), heads, kv, dim, scale, window, ctx, cache, softcap=cap, keep_first=keep)
    close(got.view(ctx.n_tokens, heads, dim), torch.cat(want), tol)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("decoding", [False, True])
@pytest.mark.parametrize("dim,page,window,keep", [(32, 16, 100, 5), (16, 8, 40, 70), (64, 32, 33, 32), (32, 64, 65, 1)])
def test_one_planted_key_is_found_exactly_where_the_window_and_the_kept_positions_let_it_be(backend, decoding, dim, page, window, keep):
    """One key is made to stand out for one query, and its value is the only one that is not zero.  It lies just inside the window, one further out, at the last kept position, one behind it, at
    position 0, at page borders, hundreds of positions back, and one ahead of the query."""
    k, dev, dtype, tol = setup(backend)
    heads, kv = 2, 1
    u = torch.zeros(dim)
    u[3] = 1.0
    mask = {"size": window, "keep_first": keep}
    cases = set()
    for qpos in (799, 640, keep + window - 1, keep + window, keep + window + 1):
        for key in (qpos, qpos - window + 1, qpos - window, keep - 1, keep, 0, page, page - 1, qpos - 1, qpos // page * page, 300):
            if 0 <= key <= qpos:
                cases.add((qpos, key))
    for qpos, key in sorted(cases):
        seen = bool(plain.visible(qpos + 1, mask)[qpos, key])
        L = qpos + 1
        first = qpos if decoding else max(0, qpos - 40)
        n = L - first
        ctx, table, n_pages, runs = step_context(dev, [(first, n)], page, k)
        cache = empty_cache(dev, dtype, n_pages, kv, page, dim, dim, table)
        keys = 0.05 * rnd(torch.Generator().manual_seed(key), L, kv, dim).float()
        keys[key, 0] = 12.0 * u
        values = torch.zeros(L, kv, dim)
        values[key, 0, 2] = 1.0                         # the result shows the weight the planted key was given
        fill_cache_by_pages(cache, table.cpu(), keys, values, page, 0)
        qkv = torch.zeros(n, (heads + 2 * kv) * dim, dtype=dtype)
        qkv[-1, :dim] = (12.0 * u).to(dtype)            # head 0 of the last token asks for the planted key
        got = k.paged_attention(qkv.to(dev), heads, kv, dim, 1.0, window, ctx, cache, softcap=40.0, keep_first=keep)
        weight = float(got.view(n, heads, dim)[-1, 0, 2])
        assert weight > 0.99 if seen else weight == 0.0, (qpos, key, weight)


@pytest.mark.gpu
@pytest.mark.parametrize("n_seqs,mode", [(4, 2), (40, 0), (130, 1)])
@pytest.mark.parametrize("window,keep", [(None, 0), (2100, 90)])
def test_capped_scores_where_decode_attention_splits_the_keys(n_seqs, mode, window, keep):
    """Long contexts in bfloat16, merged in all three ways; with kept positions the runs of tiles are dealt over what a
    query passes, which is not where the keys lie."""
    k, dev, dtype, tol = setup("hip-bf16")
    heads, kv, dim, page, scale, cap = 8, 2, 64, 16, 0.11, 3.0
    lengths = [(2500, 1100, 3000, 600, 1591, 2049)[i % 6] for i in range(n_seqs)]
    ctx, table, n_pages, runs = step_context(dev, [(L - 1, 1) for L in lengths], page, k)
    lib = k._attn_lib(dim, forms=True)
    splits = lib.sia_attn_decode_max_splits(max(lengths), lib.sia_attn_decode_walk(window or 0, keep, page))
    assert splits > 1 and lib.sia_attn_decode_mode(n_seqs, heads, kv, splits) == mode
    cache = empty_cache(dev, dtype, n_pages, kv, page, dim, dim, table)
    qkv = torch.zeros(n_seqs, (heads + 2 * kv) * dim, dtype=dtype)
    want = []
    for s, (first, n) in enumerate(runs):
        g = torch.Generator().manual_seed(s)
        L = first + 1
        keys, values = rnd(g, L, kv, dim).to(dtype), rnd(g, L, kv, dim).to(dtype)
        q = rnd(g, 1, heads, dim, std=4.0).to(dtype)
        fill_cache_by_pages(cache, table.cpu(), keys, values, page, s)
        qkv[s, :heads * dim] = q.reshape(-1)
        idx = torch.arange(L) if window is None else torch.cat([torch.arange(min(keep, max(0, first - window + 1))),
                                                                torch.arange(max(0, first - window + 1), L)])
        want.append(plain_scores(q, keys[idx], values[idx], [len(idx) - 1], scale, cap, None))
    got = k.paged_attention(qkv.to(dev), heads, kv, dim, scale, window, ctx, cache, softcap=cap, keep_first=keep)
    close(got.view(n_seqs, heads, dim), torch.cat(want), tol)


@pytest.mark.gpu
@pytest.mark.parametrize("heads,kv,dim", [(16, 4, 64), (4, 2, 144), (4, 2, 256)])
@pytest.mark.parametrize("first,n", [(0, 2048), (0, 4096), (0, 9216), (7000, 1024), (100, 700)])
def test_capped_scores_and_kept_positions_in_every_shape_of_prefill_workgroup(first, n, heads, kv, dim):
    """Long prompts and portions over a long past in bfloat16 with a window and kept positions: every shape of workgroup
    leaves out the keys in between.  The plain computation runs in float64 on the GPU."""
    if dim > 128 and n > 3000:
        pytest.skip("large heads have one shape")
    k, dev, dtype, tol = setup("hip-bf16")
    page, scale, cap, window, keep = 16, 0.09, 4.0, 700, 75
    L = first + n
    ctx, table, n_pages, runs = step_context(dev, [(first, n)], page, k)
    cache = empty_cache(dev, dtype, n_pages, kv, page, dim, dim, table)
    g = torch.Generator().manual_seed(n)
    keys, values, q = rnd(g, L, kv, dim).to(dtype), rnd(g, L, kv, dim).to(dtype), rnd(g, n, heads, dim, std=1.5).to(dtype)
    fill_cache_by_pages(cache, table.cpu(), keys, values, page, 0)
    qkv = torch.zeros(n, (heads + 2 * kv) * dim, dtype=dtype)
    qkv[:, :heads * dim] = q.reshape(n, -1)
    got = k.paged_attention(qkv.to(dev), heads, kv, dim, scale, window, ctx, cache, softcap=cap, keep_first=keep).view(n, heads, dim)
    qpos, kpos = torch.arange(first, L, device=dev)[:, None], torch.arange(L, device=dev)[None, :]
    seen = (kpos <= qpos) & ((qpos - kpos < window) | (kpos < keep))
    for h in range(heads):
        s = plain.soft_cap((q[:, h].to(dev).double() @ keys[:, h // (heads // kv)].to(dev).double().T) * scale, cap)
        want = plain.weights_over(s, seen) @ values[:, h // (heads // kv)].to(dev).double()
        assert float((got[:, h].double() - want).abs().max()) <= tol * float(want.abs().max()), h


# ---------------------------------------------------------------------------------------------------------------
def attention_part(k, dev, dtype, g, hidden, mx, value_mix):
    mask = mx.get("mask") or {}
    part = MIXERS.get("attention")({
        "hidden_size": hidden, "num_heads": mx["heads"], "num_kv_heads": mx["kv_heads"], "head_dim": mx["dim"],
        "value_head_dim": mx["vdim"], "scale": mx["scale"], "softcap": mx.get("softcap"), "window": mask.get("size"),
        "keep_first": mask.get("keep_first", 0), "out_gate": "element", "value_mix": value_mix,
        "position": {"kind": "none", "params": {}}}, env_for(k, dev, dtype))
    T = bind_part(part, g, dev, dtype, {"gate": "m.g", "value_mix": "m.vmix"}, value_mix=torch.tensor(0.35))
    return part, T


def drive(part, dev, k, h, takes, page, shared=None):
    """The part over one sequence in steps of the given sizes; ``shared(lo, hi)`` gives a step's given values."""
    need, n = part.cache_need(), h.shape[0]
    pages = -(-n // page) + 1
    table = torch.arange(pages - 1, -1, -1, dtype=torch.int32, device=dev).view(1, pages).contiguous()
    cache = empty_cache(dev, h.dtype, pages, need.num_kv_heads, page, need.head_dim, need.value_dim, table)
    outs, left, at = [], [], 0
    for take in takes:
        ctx, _, _, _ = step_context(dev, [(at, take)], page, k)
        cache.block_table = table
        ctx.shared = {} if shared is None else {"given_values": shared(at, at + take)}
        outs.append(done(part.forward(h[at:at + take].contiguous(), ctx, cache)))
        left.append(ctx.shared.get("given_values"))
        at += take
    assert at == n
    return torch.cat(outs), left


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("mx,page", [
    (dict(heads=4, kv_heads=2, dim=24, vdim=16, scale=0.3, softcap=5.0, mask={"size": 11, "keep_first": 3}), 8),
    (dict(heads=3, kv_heads=1, dim=16, vdim=40, scale=0.4, mask={"size": 30, "keep_first": 0}), 16),
    (dict(heads=4, kv_heads=4, dim=64, vdim=64, scale=0.1, softcap=2.0, mask={"size": 40, "keep_first": 18}), 16),
    (dict(heads=2, kv_heads=2, dim=10, vdim=14, scale=0.5, softcap=30.0), 16),
    (dict(heads=1, kv_heads=1, dim=128, vdim=32, scale=0.09, softcap=6.0, mask={"size": 1, "keep_first": 1}), 16)])
def test_attention_without_positions_gated_by_element_with_values_from_an_earlier_layer(backend, mx, page):
    """A prompt in portions and decoded tokens: the layer that gives its values, and one that takes them (what it caches
    is the mixture: a later step reads it back) against the plain function over the whole sequence."""
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(mx["dim"])
    hidden, n = 64, 93
    takes = [17, 2, 30, 1, 1, 9] + [1] * 33
    h, h64 = lowered(rnd(g, n, hidden), dtype, dev)
    part, T = attention_part(k, dev, dtype, g, hidden, mx, "gives")
    got, left = drive(part, dev, k, h, takes, page)
    want, v = plain.capped_attention(h64, T, "m", mx)
    close(got, want, tol * 3)
    given = torch.cat([t.clone() for t in left])
    close(given, v.reshape(n, -1), tol * 3)      # left as projected, before anything else
    other, To = attention_part(k, dev, dtype, g, hidden, mx, "takes")
    wide, wide64 = lowered(rnd(g, n, mx["kv_heads"] * mx["vdim"] + 5, std=2.0), dtype, dev)     # columns of a wider matrix
    got, _ = drive(other, dev, k, h, takes, page, shared=lambda lo, hi: wide[lo:hi, 5:])
    first = wide64[:, 5:].reshape(n, mx["kv_heads"], mx["vdim"])
    want, mixed = plain.capped_attention(h64, To, "m", mx, first)
    close(got, want, tol * 3)
    assert float((mixed - plain.lin(h64, To, "m.v").reshape(mixed.shape)).abs().max()) > 0.1     # the mixture is felt


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("heads,own,wide,extra", [(3, 20, 32, 4), (4, 64, 64, 8), (2, 7, 16, 1), (8, 32, 48, 0)])
def test_a_gate_on_every_element_of_the_heads(backend, heads, own, wide, extra):
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(own)
    for n in (1, 6, 50):
        x, x64 = lowered(rnd(g, n, heads * wide), dtype, dev)
        z, z64 = lowered(rnd(g, n, heads * own + extra, std=2.0), dtype, dev)
        got = k.element_gate(x, z[:, extra:], heads)
        want = x64.view(n, heads, wide)[:, :, :own].reshape(n, -1) * torch.sigmoid(z64[:, extra:])
        assert tuple(got.shape) == (n, heads * own)
        close(got, want, tol)


# ---------------------------------------------------------------------------------------------------------------
def latent_part(k, dev, dtype, g, hidden, mx, std=0.2):
    part = MIXERS.get("latent_attention")({
        "hidden_size": hidden, "num_heads": mx["heads"], "head_dim": mx["dim"], "rot_dim": mx["rot_dim"],
        "value_head_dim": mx["vdim"], "q_rank": mx["q_rank"], "kv_rank": mx["kv_rank"], "scale": mx["scale"], "norm_eps": 1e-5,
        "window": (mx.get("mask") or {}).get("size"), "out_gate": "element",
        "position": {"kind": "rope", "params": {"rotary_dim": mx["rot"]["dims"], "theta": mx["rot"]["base"], "scaling": None,
                                                "angles": "float64"}}}, env_for(k, dev, dtype))
    names = {"dq_norm": "m.dq.norm", "dkv_norm": "m.dkv.norm", "gate": "m.g"}
    return part, bind_part(part, g, dev, dtype, names, std=std)


LATENTS = [
    dict(heads=3, dim=16, rot_dim=8, vdim=24, q_rank=20, kv_rank=40, scale=0.2, rot={"base": 10000.0, "dims": 8}, mask={"size": 13}),
    dict(heads=1, dim=24, rot_dim=16, vdim=40, q_rank=16, kv_rank=24, scale=0.3, rot={"base": 1000.0, "dims": 8}, mask={"size": 1}),
    dict(heads=4, dim=64, rot_dim=32, vdim=64, q_rank=64, kv_rank=96, scale=0.11, rot={"base": 50000.0, "dims": 32}, mask={"size": 50}),
    dict(heads=5, dim=12, rot_dim=6, vdim=20, q_rank=14, kv_rank=22, scale=0.3, rot={"base": 777.0, "dims": 4}),
    dict(heads=24, dim=16, rot_dim=16, vdim=16, q_rank=32, kv_rank=48, scale=0.15, rot={"base": 10000.0, "dims": 16}, mask={"size": 64}),
    dict(heads=2, dim=32, rot_dim=32, vdim=40, q_rank=24, kv_rank=288, scale=0.05, rot={"base": 10000.0, "dims": 32}, mask={"size": 33}),
]


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("mx,page", list(zip(LATENTS, [8, 16, 16, 4, 16, 16])))
def test_windowed_latent_attention_with_half_pairing_and_a_gate(backend, mx, page):
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(mx["kv_rank"])
    hidden, n = 72, 141
    part, T = latent_part(k, dev, dtype, g, hidden, mx)
    h, h64 = lowered(rnd(g, n, hidden), dtype, dev)
    got, _ = drive(part, dev, k, h, [37, 2, 50, 1, 1, 9] + [1] * 41, page)
    close(got, plain.latent_attention(h64, T, "m", mx, 1e-5), tol * 3)


@pytest.mark.parametrize("backend", [b for b in BACKENDS if "bf16" not in str(b)])
@pytest.mark.parametrize("which", ["latent", "attention"])
def test_a_key_at_the_edge_of_what_a_mixer_sees(backend, which):
    """One position's input is replaced by a far larger one: a query ``window - 1`` places later gives another result, a
    query ``window`` places later gives what it gave before, unless the position is among the kept first ones, in a
    prompt and in decoding, with the position at a page's last and first place, in the middle of one, and on both sides
    of the kept positions' edge."""
    k, dev, dtype, tol = setup(backend)
    window, page, hidden, n, keep = 21, 8, 32, 70, 10
    g = torch.Generator().manual_seed(2)
    if which == "latent":
        keep = 0
        mx = dict(heads=2, dim=16, rot_dim=8, vdim=16, q_rank=16, kv_rank=32, scale=0.3, rot={"base": 1000.0, "dims": 8}, mask={"size": window})
        part, T = latent_part(k, dev, dtype, g, hidden, mx)
        whole = lambda x: plain.latent_attention(x, T, "m", mx, 1e-5)
    else:
        mx = dict(heads=2, kv_heads=1, dim=16, vdim=16, scale=0.3, softcap=3.0, mask={"size": window, "keep_first": keep})
        part, T = attention_part(k, dev, dtype, g, hidden, mx, None)
        whole = lambda x: plain.capped_attention(x, T, "m", mx)[0]
    for planted in (0, 9, 10, 15, 16, 40):
        base = rnd(g, n, hidden, std=0.3)
        other = base.clone()
        other[planted] = 8.0 * rnd(g, hidden)
        inside, outside = planted + window - 1, planted + window
        for prefix in (n, 12):                                   # all as one prompt; or a short prompt and decoding
            rows = []
            for inputs in (base, other):
                h, h64 = lowered(inputs, dtype, dev)
                out, _ = drive(part, dev, k, h, [prefix] + [1] * (n - prefix), page)
                rows.append(out.double().cpu())
                close(rows[-1], whole(h64), 3e-5)
            size = float(rows[0].abs().max())
            assert float((rows[0][inside] - rows[1][inside]).abs().max()) > 1e-3 * size
            far = float((rows[0][outside:] - rows[1][outside:]).abs().max())
            assert (far > 1e-3 * size) if planted < keep else (far <= 1e-6 * size), planted
            assert planted == 0 or float((rows[0][:planted] - rows[1][:planted]).abs().max()) == 0.0


# ---------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("page,window,keep", [(4, 10, 3), (4, 10, 4), (4, 10, 5), (8, 3, 30), (16, 40, 1), (8, 16, 0)])
def test_pages_of_kept_positions_stay_and_the_promise_covers_them(page, window, keep):
    layout = CacheLayout(kv_groups=[PagedKVNeed(1, 8, window, None, None, keep)], kv_slabs=[1], run_kv=[(0, 0)])
    cache = CacheManager(layout, page_size=page, num_pages=64, max_running=2, dtype=torch.float32, device="cpu", allocate_storage=False)
    group = cache.groups[0]
    for chunk in (1, 7, 20):
        total = 200
        cache.admit(1, total, chunk)
        promised = group.pages_to_reserve(total, chunk)
        assert 64 - group.pool.n_unpromised == promised
        at, most = 0, 0
        while at < total:
            n = min(chunk, total - at)
            cache.extend(1, n)
            table = cache.table(0, 1)
            for pos in range(at, at + n):          # whatever a query of this step sees has a page
                for j in [*range(min(keep, pos + 1)), *range(max(0, pos - window + 1), pos + 1)]:
                    assert table[j // page] >= 0, (pos, j)
            at += n
            most = max(most, len([p for p in table if p >= 0]))
            cache.check()
        assert most <= promised
        assert all(p < 0 for p in table[-(-keep // page):max(0, total - n - window + 1) // page])
        cache.release(1)
        assert group.pool.n_free == 64
