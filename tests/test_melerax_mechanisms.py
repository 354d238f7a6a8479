"""Every mechanism of the Melerax design alone: the kernel (its torch twin on the CPU, the HIP kernel on the GPU in
float32 and bfloat16) against the plain implementation's function for it, at sizes of all kinds."""

import types

import pytest
import torch

import plain_melerax as plain
from simple_inference_amd.parts import FEED_FORWARDS, MIXERS, NORMS
from simple_inference_amd.parts.context import LayerCache, NormedSum, ResidualStream
from test_famepel_mechanisms import done, f32, portions, rounded, rows_of
from test_feduzen_mechanisms import empty_cache, fill_cache_by_pages, step_context
from test_lunerax_mechanisms import bind_part, env_for
from test_mogisun_mechanisms import BACKENDS, close, lowered, rnd, setup


def batch(dev, step, slots, tables=None, page=16, ids=None):
    """The step function's layout of a step ``[(sequence, first position, tokens)]``; ``tables``: every sequence's pages."""
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)
    q = [n for _, _, n in step]
    cu = [sum(q[:i]) for i in range(len(q) + 1)]
    ctx = types.SimpleNamespace(
        n_tokens=cu[-1], n_seqs=len(step), positions=i32([a + i for _, a, n in step for i in range(n)]),
        seq_of_token=i32([s for s, n in enumerate(q) for _ in range(n)]), cu_q=i32(cu), kv_len=i32([a + n for _, a, n in step]),
        state_slots=i32([slots[s] for s, _, _ in step]), max_q_len=max(q), max_kv_len=max(a + n for _, a, n in step),
        n_decode_seqs=sum(n == 1 for n in q), q_lens=q, kv_bound=0, extra={},
        max_run_kv_len=max([a + n for _, a, n in step if n > 1], default=0))
    if ids is not None:
        ctx.token_ids = i32([t for s, a, n in step for t in ids[s][a:a + n]])
    table = None
    if tables is not None:
        width = max(len(t) for t in tables)
        table = i32([tables[s] + [-1] * (width - len(tables[s])) for s, _, _ in step])
    return ctx, table


def scrambled(lengths, page):
    pages = torch.randperm(sum(-(-n // page) for n in lengths), generator=torch.Generator().manual_seed(5)).tolist()
    return [[pages.pop() for _ in range(-(-n // page))] for n in lengths]


# ---------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("pairs,hidden,scale", [((61, 7, 5), 40, 1.0), ((1, 3, 1), 96, 2.5), ((509, 2147483647, 2147483646), 33, 1.0),
                                                ((8, 0, 1), 64, 1.0), ((8, 1, 0), 64, 1.0)])
def test_pairs_of_tokens_over_any_cut_and_a_new_sequence_in_an_old_slot(backend, pairs, hidden, scale):
    """The token before a step's first one comes from the slot; a sequence's first token takes the last row whatever the
    slot's last holder left."""
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(hidden)
    vocab = 53
    table, table64 = lowered(rnd(g, vocab, hidden), dtype, dev)
    second, second64 = lowered(rnd(g, pairs[0] + 1, hidden), dtype, dev)
    lengths, slots = [38, 6, 22], [4, 0, 2]
    ids = [torch.randint(0, vocab, (n,), generator=g).tolist() for n in lengths]
    state = torch.full((6, 1), 17, dtype=torch.int32, device=dev)
    cfg = dict(zip(("buckets", "mul_prev", "mul_cur"), pairs))
    want = [table64[t] * scale + second64[plain.pair_rows(t, cfg)] for t in ids]
    for step in portions(lengths, [2, 1, 9, 1, 3, 17]):
        ctx, _ = batch(dev, step, slots, ids=ids)
        got = k.embed_pairs(ctx.token_ids, table, second, pairs, ctx, state, scale=scale)
        close(got, torch.cat([want[s][a:a + n] for s, a, n in step]), 2e-6)
    assert state[:, 0].tolist() == [ids[1][-1], 17, ids[2][-1], 17, ids[0][-1], 17]


# ---------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width", [96, 50, 176, 1024, 2056, 8200])
def test_norm_behind_a_sublayer_with_its_scale_its_bias_and_two_inner_norms(backend, width):
    """``x += N(y + b) * s`` and ``x += N(f1 rms(y1) g1 + f2 rms(y2) g2) * s`` through the norm part, and the inner sum alone
    of one, two and three terms."""
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(width)
    n, eps, inner = 7, 3e-4, 1e-2
    norm = NORMS.get("rmsnorm")({"size": width, "eps": eps, "unit_offset": True, "scaled": True}, env_for(k, dev, dtype))
    w, s = rnd(g, width, std=0.3), 1 + rnd(g, width, std=0.3)
    norm.bind({"weight": f32(w, dev), "scale": f32(s, dev)})
    res = rnd(g, n, width, std=2.0)
    y, y64 = lowered(rnd(g, n, width, std=0.05), dtype, dev)       # small: the eps inside the root weighs
    b = rnd(g, width, std=0.05)
    stream = ResidualStream(f32(res, dev))
    from simple_inference_amd.parts.context import BiasedDelta
    low = norm.add_normed(stream, BiasedDelta(y, f32(b, dev), k))
    want = rounded(res) + plain.offset_norm(y64 + rounded(b), rounded(w), eps) * rounded(s)
    close(stream.residual, want, 3e-6)
    assert low.dtype == dtype and torch.equal(low.float(), stream.residual.to(dtype).float())
    ys = [lowered(rnd(g, n, width, std=std), dtype, dev) for std in (0.1, 1.5, 0.4)]
    gains = [1 + rnd(g, width, std=0.3) for _ in ys]
    factors = (0.5, -1.25, 2.0)
    term = lambda i: (ys[i][0], factors[i], f32(gains[i], dev), inner)
    plain_term = lambda i: factors[i] * plain.rms(ys[i][1], inner) * rounded(gains[i])
    stream = ResidualStream(f32(res, dev))
    low = norm.add_normed(stream, NormedSum([term(0), term(1)], k))
    want = rounded(res) + plain.offset_norm(plain_term(0) + plain_term(1), rounded(w), eps) * rounded(s)
    close(stream.residual, want, 3e-6)
    assert torch.equal(low.float(), stream.residual.to(dtype).float())
    for count in (1, 2, 3):
        close(NormedSum([term(i) for i in range(count)], k).compute(), sum(plain_term(i) for i in range(count)), tol)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("n,width,inter", [(5, 64, 40), (33, 128, 72), (19, 50, 27), (1, 192, 96), (16, 128, 1000)])
def test_the_gelu_gate_with_biases(backend, n, width, inter):
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(n)
    part = FEED_FORWARDS.get("swiglu")({"hidden_size": width, "intermediate_size": inter, "activation": "gelu_tanh", "bias": True},
                                       env_for(k, dev, dtype))
    T = bind_part(part, g, dev, dtype, {f"{m}_bias": f"m.{m}.b" for m in ("gate", "up", "down")}, std=0.2)
    h, h64 = lowered(rnd(g, n, width), dtype, dev)
    close(done(part.forward(h, None)), plain.gated_dense(h64, T, "m"), tol * 2)
    assert part.plain_form() is None       # a kernel that runs whole blocks with the silu gate must leave this one alone
    with pytest.raises(ValueError):
        FEED_FORWARDS.get("swiglu")({"hidden_size": 8, "intermediate_size": 8, "bias": True}, env_for(k, dev, dtype))


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("experts,top,width", [(8, 2, 96), (5, 5, 50), (64, 6, 128), (1, 1, 40)])
def test_the_routers_bias_takes_part_in_the_choice_and_the_weights(backend, experts, top, width):
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(experts)
    n = 19
    h, h64 = lowered(rnd(g, n, width), dtype, dev)
    R, bias = rnd(g, experts, width, std=width ** -0.5), rnd(g, experts)
    bias[experts - 1] += 20.0                     # one expert is chosen by its bias alone
    T = {"m.router": rounded(R), "m.router.b": rounded(bias)}
    ids, weights = k.moe_route(h, f32(R, dev), top, bias=f32(bias, dev))
    got = torch.zeros(n, experts, dtype=torch.float64).scatter(1, ids.long().cpu(), weights.double().cpu())
    close(got, plain.routing(h64, T, "m", top), 2e-5)
    assert bool((ids[:, 0] == experts - 1).all())
    close(weights.sum(-1), torch.ones(n), 1e-5)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("experts,top,width,ff,shared,n", [(4, 2, 96, 32, 40, 5), (8, 8, 64, 96, None, 40), (3, 1, 50, 18, 22, 33),
                                                           (6, 2, 128, 64, 64, 90), (1, 1, 32, 32, 1, 70)])
def test_experts_without_a_gate_slot_by_slot_and_in_tiles(backend, experts, top, width, ff, shared, n):
    """The part as the plan builds it; the tokens' logits lie far apart, so that rounding changes nobody's choice."""
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(n)
    part = FEED_FORWARDS.get("moe")({"hidden_size": width, "experts": experts, "top": top, "expert_size": ff, "activation": "gelu",
                                     "router_bias": True, "shared_size": shared, "shared_gate": False}, env_for(k, dev, dtype))
    names = {"router_bias": "m.router.b", "shared_up": "m.shared.up", "shared_down": "m.shared.down"}
    names.update({f"{w}{e}": f"m.e{e}.{w}" for e in range(experts) for w in ("up", "down")})
    T = bind_part(part, g, dev, dtype, names, std=0.15, router=rnd(g, experts, width, std=3.0), router_bias=rnd(g, experts))
    h, h64 = lowered(rnd(g, n, width), dtype, dev)
    mlp = {"router": {"experts": experts, "top": top}, "shared": shared}
    close(part.forward(h, None), plain.routed_experts(h64, T, "m", mlp), tol * 2)


# ---------------------------------------------------------------------------------------------------------------
ROWS = [  # heads, kv heads, dim, vdim, taps, rotated, pairing, norm over, page width, page size
    (4, 2, 24, 16, 3, 8, "interleaved", "row", None, 8), (1, 1, 8, 8, 1, 8, "interleaved", "row", 16, 16),
    (6, 3, 48, 96, 3, 48, "interleaved", "row", 96, 16), (3, 1, 10, 14, 5, 6, "interleaved", "row", 16, 16),
    (5, 5, 7, 9, 2, 4, "half", "head", None, 4), (8, 2, 64, 64, 4, 64, "half", "head", None, 32),
    (2, 1, 144, 40, 16, 2, "interleaved", None, 160, 16), (32, 8, 128, 128, 4, 128, "interleaved", "row", None, 16),
    (2, 2, 16, 24, 2, 0, "half", "row", 32, 8)]


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("heads,kv,dim,vdim,taps,rot,pairing,over,wide,page", ROWS)
def test_convolved_rows_are_normed_turned_and_put_into_the_pages_through_any_cut(backend, heads, kv, dim, vdim, taps, rot, pairing,
                                                                                 over, wide, page):
    """Three sequences of unequal length in scattered slots and pages: the queries, and every key and value in its page,
    are the plain functions' over the whole sequence.  q, k and v are columns of a wider matrix, behind one another with
    gaps; the ring lies at the front of a longer state row."""
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(heads * 100 + dim)
    lengths, slots = [70, 6, 41], [4, 0, 2]
    sizes = (heads * dim, kv * dim, kv * vdim)
    up8 = lambda x: x + (-x) % 8
    cols = (8, 8 + up8(sizes[0]), 8 + up8(sizes[0]) + up8(sizes[1]))
    width = cols[2] + up8(sizes[2]) + 16
    rows = [lowered(rnd(g, n, width), dtype, dev) for n in lengths]
    channels = sum(sizes)
    bias, conv = rnd(g, channels, std=0.5), rnd(g, channels, taps, std=0.6)
    gains = [1 + rnd(g, s, std=0.3) for s in ((sizes[0], sizes[1]) if over == "row" else (dim, dim))]
    eps, base = 1e-3, 300.0
    freq = base ** (-2.0 * torch.arange(rot // 2, dtype=torch.float64) / max(rot, 1))
    angles = torch.arange(128, dtype=torch.float64)[:, None] * freq
    cos, sin = (f32(angles.cos(), dev), f32(angles.sin(), dev)) if rot else (None, None)

    def reference(x64):
        u = torch.cat([x64[:, c:c + s] for c, s in zip(cols, sizes)], 1) + rounded(bias)
        q, kk, v = plain.causal_conv(u, rounded(conv)).split(sizes, 1)
        out = []
        for x, h, gain in ((q, heads, gains[0]), (kk, kv, gains[1])):
            if over == "row":
                x = (plain.rms(x, eps) * rounded(gain)).reshape(-1, h, dim)
            else:
                x = x.reshape(-1, h, dim)
                x = plain.rms(x, eps) * rounded(gain) if over else x
            if rot and pairing == "interleaved":
                x = plain.rotate_pairs(x, {"base": base, "dims": rot})
            elif rot:
                n = x.shape[0]
                c, s = angles[:n].cos()[:, None], angles[:n].sin()[:, None]
                a, b = x[..., :rot // 2], x[..., rot // 2:rot]
                x = torch.cat([a * c - b * s, b * c + a * s, x[..., rot:]], -1)
            out.append(x)
        return out[0], out[1], v.reshape(-1, kv, vdim)

    want = [reference(x64) for _, x64 in rows]
    tables = scrambled(lengths, page)
    n_pages = sum(len(t) for t in tables)
    cache = empty_cache(dev, dtype, n_pages, kv, page, wide or dim, wide or vdim, None)
    tail = 3
    state = torch.zeros(6, taps * channels + tail, dtype=torch.float32, device=dev)
    state[:, taps * channels:] = 3.0
    cache.state = state[:, :taps * channels]
    norm = (f32(gains[0], dev), f32(gains[1], dev), eps, over) if over else None
    for step in portions(lengths, [2, 1, 9, 1, 3, 37]):
        ctx, cache.block_table = batch(dev, step, slots, tables, page)
        proj = torch.cat([rows[s][0][a:a + n] for s, a, n in step]).contiguous()
        got = k.row_prepare(proj[:, :width - 8], cols, heads, kv, dim, vdim, rot, cos, sin, pairing, f32(bias, dev),
                            f32(conv.t().contiguous(), dev), norm, wide, ctx, cache).view(ctx.n_tokens, heads, wide or dim)
        close(got[..., :dim], torch.cat([want[s][0][a:a + n] for s, a, n in step]), tol)
        assert float(got[..., dim:].abs().max()) == 0.0 if (wide or dim) > dim else True
    for s, n in enumerate(lengths):
        for p in range(n):
            pg, off = tables[s][p // page], p % page
            close(cache.k_pages[pg, :, off, :dim], want[s][1][p], tol)
            close(cache.v_pages[pg, :, :vdim, off], want[s][2][p], tol)
    if wide:
        assert float(cache.k_pages[..., dim:].abs().max() if wide > dim else 0.0) == 0.0
        assert float(cache.v_pages[:, :, vdim:].abs().max() if wide > vdim else 0.0) == 0.0
    assert float(state[[1, 3, 5], :taps * channels].abs().max()) == 0.0
    assert float((state[:, taps * channels:] - 3.0).abs().max()) == 0.0      # what lies behind the ring is not its own


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("heads,kv,dim,block,cap,page", [(3, 3, 32, 24, 2.0, 8), (4, 2, 16, 20, None, 16), (8, 2, 64, 37, 1.5, 16),
                                                         (4, 4, 128, 64, 4.0, 16), (2, 1, 144, 33, 2.0, 32), (16, 1, 32, 50, 2.0, 16),
                                                         (2, 2, 24, 18, 6.0, 4), (6, 3, 96, 120, 30.0, 16), (2, 1, 16, 1, 3.0, 8)])
def test_capped_scores_inside_blocks_in_prompts_and_decoding(backend, heads, kv, dim, block, cap, page):
    """A whole prompt, portions that begin inside blocks and at their edges, single tokens at a block's first, second and
    last place.  Pages of finished blocks have no entry in the block table."""
    k, dev, dtype, tol = setup(backend)
    scale, T = 0.31, 400
    runs = [(0, T), (block + 3, 2 * block + 1), (300, 60), (block, 1), (block + 1, 1), (2 * block - 1, 1), (3 * page, 1), (0, 1),
            (399, 1), (200, 2), (4 * block - 1, 2)]
    ctx, table, n_pages, runs = step_context(dev, runs, page, k)
    cache = empty_cache(dev, dtype, n_pages, kv, page, dim, dim, table)
    qkv = torch.zeros(ctx.n_tokens, heads * dim, dtype=dtype)
    g = torch.Generator().manual_seed(dim)
    want, row = [], 0
    held = table.clone()
    for s, (first, n) in enumerate(runs):
        L = first + n
        keys, values = rnd(g, L, kv, dim).to(dtype), rnd(g, L, kv, dim).to(dtype)
        q = rnd(g, n, heads, dim).to(dtype)
        fill_cache_by_pages(cache, table.cpu(), keys, values, page, s)
        qkv[row:row + n] = q.reshape(n, heads * dim)
        seen = plain.visible(L, {"size": block})[first:]
        out = []
        for h in range(heads):
            scores = plain.soft_cap((q[:, h].double() @ keys[:, h // (heads // kv)].double().T) * scale, cap)
            out.append(torch.softmax(scores.masked_fill(~seen, float("-inf")), -1) @ values[:, h // (heads // kv)].double())
        want.append(torch.stack(out, 1))
        held[s, :first // block * block // page] = -1
        row += n
    cache.block_table = held
    got = k.paged_attention(qkv.to(dev), heads, kv, dim, scale, None, ctx, cache, chunk=block, softcap=cap)
    close(got.view(ctx.n_tokens, heads, dim), torch.cat(want), tol)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("decoding", [False, True])
@pytest.mark.parametrize("dim,page,block", [(32, 16, 100), (16, 8, 40), (64, 32, 33), (32, 64, 65)])
def test_one_planted_key_is_found_exactly_inside_its_block(backend, decoding, dim, page, block):
    """One key stands out for one query, and its value is the only one that is not zero: the query finds it at its block's
    first position and right before itself, and not at the last position of the block before, hundreds of positions back,
    or one ahead."""
    k, dev, dtype, tol = setup(backend)
    heads, kv, cap = 2, 1, 50.0
    u = torch.zeros(dim)
    u[3] = 6.0
    value = torch.linspace(-1, 1, dim)
    for query in (4 * block, 4 * block + 1, 5 * block - 1, 3 * block + block // 2):
        start = query // block * block
        places = {start, start - 1, start + 1, query, query - 1, 0, page, page - 1, query + 1, start - block}
        for at in sorted(p for p in places if 0 <= p <= query + 1):
            L = query + (1 if decoding else 2)
            if at >= L:
                continue
            runs = [(query, 1)] if decoding else [(0, L)]
            ctx, table, n_pages, runs = step_context(dev, runs, page, k)
            cache = empty_cache(dev, dtype, n_pages, kv, page, dim, dim, table)
            keys, values = torch.zeros(L, kv, dim), torch.zeros(L, kv, dim)
            keys[at, 0], values[at, 0] = u, value
            fill_cache_by_pages(cache, table.cpu(), keys.to(dtype), values.to(dtype), page, 0)
            qkv = torch.zeros(ctx.n_tokens, heads * dim, dtype=dtype)
            qkv[0 if decoding else query] = u.repeat(heads).to(dtype)
            got = k.paged_attention(qkv.to(dev), heads, kv, dim, 0.5, None, ctx, cache, chunk=block, softcap=cap)
            row = got[0 if decoding else query].view(heads, dim).double().cpu()
            if start <= at <= query:
                close(row, value.expand(heads, dim), 3e-2)
            else:
                assert float(row.abs().max()) == 0.0, (query, at)


# ---------------------------------------------------------------------------------------------------------------
UNITS = [(72, 3, 4), (40, 1, 1), (64, 64, 2), (66, 2, 3), (128, 2, 4), (160, 2, 16), (384, 3, 4), (50, 5, 2), (1024, 4, 4), (80, 5, 3)]


def unit_terms(g, width, blocks, taps, dtype, dev):
    bs = width // blocks
    ra, ra64 = lowered(rnd(g, blocks, bs, bs, std=bs ** -0.5), dtype, dev)
    ri, ri64 = lowered(rnd(g, blocks, bs, bs, std=bs ** -0.5), dtype, dev)
    T = {n: rounded(rnd(g, width, std=0.5)) for n in ("y_bias", "x_bias", "conv_bias", "ra_bias", "ri_bias")}
    T["lam"], T["conv"] = rounded(rnd(g, width) - 2.0), rounded(rnd(g, width, taps, std=0.6))
    terms = {n: f32(T[n], dev) for n in ("y_bias", "x_bias", "conv_bias", "ra_bias", "ri_bias")}
    rate = 8.0 * torch.nn.functional.softplus(T["lam"], threshold=1e9)
    terms.update(conv=f32(T["conv"].t().contiguous(), dev), ra=ra, ri=ri, rate=f32(rate, dev))
    T.update(ra=ra64, ri=ri64)
    return terms, T


def unit_reference(y64, x64, T, blocks):
    u = plain.causal_conv(x64 + T["x_bias"], T["conv"]) + T["conv_bias"]
    r = plain.block_gate(u, T["ra"], T["ra_bias"].view(blocks, -1))
    i = plain.block_gate(u, T["ri"], T["ri_bias"].view(blocks, -1))
    return plain.linear_unit(u, r, i, T["lam"]) * plain.gelu_tanh(y64 + T["y_bias"])


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width,blocks,taps", UNITS)
def test_the_linear_unit_carries_its_state_through_any_cut(backend, width, blocks, taps):
    """Sequences of unequal length in scattered slots, in portions from one token to beyond two chunks of the scan, the
    batch's order changing; more single tokens at once than a workgroup takes.  The branches are columns of a wider
    matrix, the state lies at the front of a longer row."""
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(width)
    lengths = [230, 6, 131, 64] + [3] * 15
    slots = [4, 0, 2] + list(range(6, 22))
    at_x = width + (-width) % 8
    rows = [lowered(rnd(g, n, 2 * at_x + 8), dtype, dev) for n in lengths]
    terms, T = unit_terms(g, width, blocks, taps, dtype, dev)
    floats = width * (1 + (taps if taps > 1 else 0))
    state = torch.zeros(23, floats + 4 + (-floats) % 4, dtype=torch.float32, device=dev)
    state[:, floats:] = 3.0
    offsets = [sum(lengths[:s]) for s in range(len(lengths))]
    got = torch.zeros(sum(lengths), width, dtype=torch.float64)
    for step in portions(lengths, [2, 1, 64, 1, 3, 129, 1, 65]):
        ctx, _ = batch(dev, step, slots)
        proj = torch.cat([rows[s][0][a:a + n] for s, a, n in step]).contiguous()
        out = k.linear_unit(proj[:, :2 * at_x], 0, at_x, terms, blocks, ctx, state[:, :floats])
        got[rows_of(step, offsets)] = out.double().cpu()
    singles = [(s, 0, 1) for s in range(len(lengths))]      # nineteen new sequences of one token
    ctx, _ = batch(dev, singles, slots)
    fresh = torch.zeros_like(state)
    one = k.linear_unit(torch.cat([r[0][:1] for r in rows]).contiguous(), 0, at_x, terms, blocks, ctx, fresh).double().cpu()
    want = [unit_reference(x64[:, :width], x64[:, at_x:at_x + width], T, blocks) for _, x64 in rows]
    close(got, torch.cat(want), tol * 2)
    close(one, torch.cat([w[:1] for w in want]), tol * 2)
    assert float(state[[1, 3, 5, 22], :floats].abs().max()) == 0.0
    assert float((state[:, floats:] - 3.0).abs().max()) == 0.0


@pytest.mark.parametrize("backend", BACKENDS)
def test_the_linear_unit_remembers_one_token_over_hundreds(backend):
    """Built inputs: one token writes and all others do not (their inputs are zero and so is what they write); the decays
    are slow for half of the channels and fast for the other half.  After 300 tokens the slow channels hold what the decay's
    power says, the fast ones nothing, in one prompt and in single tokens."""
    k, dev, dtype, tol = setup(backend)
    width, n, blocks = 32, 310, 2
    g = torch.Generator().manual_seed(3)
    terms, T = unit_terms(g, width, blocks, 1, dtype, dev)
    zeros = torch.zeros(width, dtype=torch.float64)
    lam = torch.cat([torch.full((16,), -7.5), torch.full((16,), 1.0)]).double()
    for name in ("ra_bias", "ri_bias"):
        terms[name], T[name] = f32(zeros, dev), zeros
    for name in ("ra", "ri"):       # half-open gates
        terms[name], T[name] = torch.zeros_like(terms[name]), torch.zeros_like(T[name])
    T.update(x_bias=zeros, conv_bias=zeros, lam=lam, conv=torch.ones(width, 1, dtype=torch.float64), y_bias=zeros)
    for name in ("x_bias", "conv_bias", "y_bias"):
        terms[name] = f32(T[name], dev)
    terms["conv"] = f32(T["conv"].t().contiguous(), dev)
    terms["rate"] = f32(8.0 * torch.nn.functional.softplus(lam), dev)
    rows = torch.zeros(n, 2 * width, dtype=torch.float64)
    rows[:, :width] = 2.0
    rows[5, width:] = 3.0
    x, x64 = lowered(rows, dtype, dev)
    want = unit_reference(x64[:, :width], x64[:, width:], T, blocks)
    assert float(want[-1, :16].abs().min()) > 0.01 and float(want[-1, 16:].abs().max()) < 1e-20
    for cuts in ([(0, n)], [(0, 7), (7, 9)] + [(t, t + 1) for t in range(9, n)]):
        state = torch.zeros(2, width, dtype=torch.float32, device=dev)
        got = [k.linear_unit(x[lo:hi].contiguous(), 0, width, terms, blocks, batch(dev, [(0, lo, hi - lo)], [1])[0], state)
               for lo, hi in cuts]
        got = torch.cat(got).double().cpu()
        close(got, want, tol)
        assert float(((got - want)[-1, :16] / want[-1, :16]).abs().max()) < (2e-2 if dtype == torch.bfloat16 else 1e-4)


# ---------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width,mixtures", [(64, 5), (50, 2), (2056, 1), (1, 3)])
def test_rows_are_mixed_with_the_row_before_through_any_cut(backend, width, mixtures):
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(width)
    lengths, slots = [38, 6, 22], [4, 0, 2]
    rows = [lowered(rnd(g, n, width), dtype, dev) for n in lengths]
    mu = torch.rand(mixtures, width, generator=g, dtype=torch.float64)
    state = torch.zeros(6, width + 5, dtype=torch.float32, device=dev)
    want = [torch.stack([plain.token_shift(x64, rounded(m)) for m in mu]) for _, x64 in rows]
    for step in portions(lengths, [2, 1, 9, 1, 3, 17]):
        ctx, _ = batch(dev, step, slots)
        got = k.token_shift(torch.cat([rows[s][0][a:a + n] for s, a, n in step]).contiguous(), f32(mu, dev), ctx, state, 5)
        close(got, torch.cat([want[s][:, a:a + n] for s, a, n in step], 1), tol)
    assert float(state[:, :5].abs().max()) == 0.0 and float(state[[1, 3, 5]].abs().max()) == 0.0


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("groups,rows,last,K", [(5, 128, 16, 256), (2, 40, 40, 64), (5, 50, 7, 128), (3, 24, 60, 50), (5, 1024, 64, 192)])
@pytest.mark.parametrize("M", [1, 8, 16, 40])
def test_groups_of_rows_read_inputs_of_their_own(backend, groups, rows, last, K, M):
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(rows + M)
    x, x64 = lowered(rnd(g, groups, M, K), dtype, dev)
    w, w64 = lowered(rnd(g, (groups - 1) * rows + last, K, std=K ** -0.5), dtype, dev)
    main, low = k.grouped_linear(x, w, rows)
    for i in range(groups - 1):
        close(main[i], x64[i] @ w64[i * rows:(i + 1) * rows].T, tol)
    close(low, x64[-1] @ w64[(groups - 1) * rows:].T, tol)


WKV = [(3, 16, 10), (1, 8, 1), (2, 64, 32), (4, 128, 64), (2, 40, 16), (1, 264, 24), (5, 12, 9), (1, 200, 8)]


def wkv_reference(rkvg64, low64, T, H, D, eps):
    n = low64.shape[0]
    r, kk, v = (rkvg64[i].reshape(n, H, D) for i in range(3))
    w = torch.exp(-torch.exp(torch.tanh(low64) @ T["w2"].T + T["w0"])).reshape(n, H, D)
    o = plain.rms(plain.bonus_recurrence(r, kk, v, w, T["u"].view(H, D)), eps).reshape(n, H * D)
    return o * T["norm"] * plain.silu(rkvg64[3])


def head_close(got, want, tol, dtype):
    """As ``close`` over the rows, but for the few of bfloat16 whose head nearly cancels: the norm divides by a small
    number there, and what was rounded before it weighs many times more."""
    rows = (got.double().cpu() - want).pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()
    assert bool(torch.isfinite(rows).all())
    assert float((rows.sort().values[:max(1, int(rows.numel() * 0.95))] if dtype == torch.bfloat16 else rows).max()) <= tol


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("H,D,rank", WKV)
def test_the_state_with_a_bonus_carries_through_any_cut(backend, H, D, rank):
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(H * 1000 + D)
    lengths, slots = [78, 6, 42], [4, 0, 2]
    rows = [lowered(rnd(g, 4, n, H * D), dtype, dev) for n in lengths]
    lows = [lowered(rnd(g, n, rank), dtype, dev) for n in lengths]
    w2, w2_64 = lowered(rnd(g, H * D, rank, std=rank ** -0.5), dtype, dev)
    T = {"w2": w2_64, "w0": rounded(rnd(g, H * D) - 1.5), "u": rounded(rnd(g, H * D)), "norm": rounded(1 + rnd(g, H * D, std=0.3))}
    eps, tail = 1e-3, 5
    state = torch.zeros(6, H * D * D + tail, dtype=torch.float32, device=dev)
    state[:, H * D * D:] = 3.0
    offsets = [sum(lengths[:s]) for s in range(len(lengths))]
    got = torch.zeros(sum(lengths), H * D, dtype=torch.float64)
    for step in portions(lengths, [2, 1, 9, 1, 3, 37]):
        ctx, _ = batch(dev, step, slots)
        rkvg = torch.cat([rows[s][0][:, a:a + n] for s, a, n in step], 1).contiguous()
        low = torch.cat([lows[s][0][a:a + n] for s, a, n in step]).contiguous()
        out = k.bonus_recurrence(rkvg, low, w2, f32(T["w0"], dev), f32(T["u"], dev), f32(T["norm"], dev), H, D, eps, ctx, state)
        got[rows_of(step, offsets)] = out.double().cpu()
    want = torch.cat([wkv_reference(rows[s][1], lows[s][1], T, H, D, eps) for s in range(len(lengths))])
    head_close(got, want, tol, dtype)
    assert float(state[[1, 3, 5], :H * D * D].abs().max()) == 0.0
    assert float((state[:, H * D * D:] - 3.0).abs().max()) == 0.0      # what lies behind the matrices is not theirs


@pytest.mark.parametrize("backend", BACKENDS)
def test_the_bonus_is_for_the_current_token_only_and_channels_fade_at_their_own_rates(backend):
    """Built inputs: two key channels are written once each; one keeps nearly all of it over 300 tokens, the other loses it.
    A query along both reads both values right away (the current token's own write weighed by the bonus, which here is 3
    where the state's share is 1), and 300 tokens later the slow channel's alone."""
    k, dev, dtype, tol = setup(backend)
    H, D, n, rank = 1, 16, 320, 8
    g = torch.Generator().manual_seed(1)
    e = torch.eye(D, dtype=torch.float64)
    rkvg = torch.zeros(4, n, D, dtype=torch.float64)
    rkvg[0] = e[0] + e[1]                      # everybody asks along the first two channels
    rkvg[3] = 4.0                              # an open output gate
    for t in range(n):
        rkvg[1, t] = e[2 + t % (D - 2)]
        rkvg[2, t] = rnd(g, D)
    a, b = torch.arange(D, dtype=torch.float64) - 7.5, torch.linspace(2, -1, D, dtype=torch.float64)
    rkvg[1, 5], rkvg[2, 5] = e[0], a
    rkvg[1, 6], rkvg[2, 6] = e[1], b
    T = {"w2": torch.zeros(D, rank, dtype=torch.float64), "u": torch.full((D,), 3.0, dtype=torch.float64),
         "norm": torch.ones(D, dtype=torch.float64), "w0": torch.full((D,), -9.0, dtype=torch.float64)}
    T["w0"][1] = 1.0
    x, x64 = lowered(rkvg, dtype, dev)
    low, low64 = lowered(torch.ones(n, rank, dtype=torch.float64), dtype, dev)
    want = wkv_reference(x64, low64, T, H, D, 1e-6)
    cos = lambda p, q: float((p * q).sum() / p.norm() / q.norm())
    for cuts in ([(0, n)], [(0, 7), (7, 9)] + [(t, t + 1) for t in range(9, n)]):
        state = torch.zeros(2, D * D, dtype=torch.float32, device=dev)
        got = torch.cat([k.bonus_recurrence(x[:, lo:hi].contiguous(), low[lo:hi].contiguous(), lowered(T["w2"], dtype, dev)[0],
                                            f32(T["w0"], dev), f32(T["u"], dev), f32(T["norm"], dev), H, D, 1e-6,
                                            batch(dev, [(0, lo, hi - lo)], [1])[0], state) for lo, hi in cuts]).double().cpu()
        close(got[5:], want[5:], tol * 2)
        assert cos(got[6], a + 3.0 * b) > 0.999 and cos(got[n - 1], a) > 0.999


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("n,rank", [(1, 16), (16, 128), (64, 8), (65, 40), (200, 72), (70, 13)])
def test_decays_of_many_and_few_tokens_are_not_rounded_on_their_way(backend, n, rank):
    """The tanh's results lie close to one another and the products are large, so that rounding them to 8 bits would show
    far beyond the tolerance: the state after the step is held to the float32 tolerance in both modes."""
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(n * 100 + rank)
    H, D = 3, 24
    low, low64 = lowered(1.0 + rnd(g, n, rank, std=0.05), dtype, dev)
    w2, w2_64 = lowered(rnd(g, H * D, rank, std=2 * rank ** -0.5), dtype, dev)
    T = {"w2": w2_64, "w0": rounded(-1.0 - w2_64.sum(1) * 0.76), "u": torch.ones(H * D, dtype=torch.float64),
         "norm": torch.ones(H * D, dtype=torch.float64)}
    x, x64 = lowered(rnd(g, 4, n, H * D), dtype, dev)
    state = torch.zeros(1, H * D * D, dtype=torch.float32, device=dev)
    k.bonus_recurrence(x, low, w2, f32(T["w0"], dev), f32(T["u"], dev), f32(T["norm"], dev), H, D, 1e-5,
                       batch(dev, [(0, 0, n)], [0])[0], state)
    w = torch.exp(-torch.exp(torch.tanh(low64) @ T["w2"].T + T["w0"])).reshape(n, H, D)
    S = torch.zeros(H, D, D, dtype=torch.float64)
    for t in range(n):
        S = w[t][:, :, None] * S + x64[1, t].view(H, D, 1) * x64[2, t].view(H, 1, D)
    close(state[0].view(H, D, D), S, 3e-5)


# ---------------------------------------------------------------------------------------------------------------
def run_part(part, h, dev, cuts, slots=(1,), page=16, kv=None, dtype=None, wide=None, T=64):
    """A mixer part over one sequence in portions; pages of the part's own widths where it keeps some."""
    need, sneed = part.cache_need(), part.state_need()
    tables = [list(range(-(-h.shape[0] // page)))[::-1]]
    cache = LayerCache() if need is None else empty_cache(dev, h.dtype, len(tables[0]), need.num_kv_heads, page, need.head_dim,
                                                          need.value_dim, None)
    if sneed is not None:
        cache.state = torch.zeros(3, *sneed.shape, dtype=torch.float32, device=dev)
    outs = []
    for lo, hi in cuts:
        ctx, table = batch(dev, [(0, lo, hi - lo)], [1], tables, page)
        cache.block_table = table
        outs.append(done(part.forward(h[lo:hi].contiguous(), ctx, cache)))
    return torch.cat(outs)


CUTS = ((0, 17), (17, 19), (19, 20), (20, 21), (21, 40), (40, 41))


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("mx,hidden", [(dict(width=72, blocks=3, conv=4), 64), (dict(width=50, blocks=5, conv=1), 96),
                                       (dict(width=256, blocks=2, conv=3), 128)])
def test_the_linear_unit_part_is_the_plain_block(backend, mx, hidden):
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(11)
    part = MIXERS.get("rglru")({"hidden_size": hidden, "width": mx["width"], "blocks": mx["blocks"], "conv_taps": mx["conv"]},
                               env_for(k, dev, dtype))
    names = {f"{n}_bias": f"m.{n}.b" for n in ("y", "x", "conv", "ra", "ri")}
    T = bind_part(part, g, dev, dtype, names, std=0.2)
    h, h64 = lowered(rnd(g, 41, hidden), dtype, dev)
    close(run_part(part, h, dev, CUTS), plain.recurrent_block(h64, T, "m"), tol * 2)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("heads,dim,rank,hidden", [(3, 16, 10, 64), (2, 64, 32, 128), (1, 24, 1, 50)])
def test_the_wkv_part_is_the_plain_mixer(backend, heads, dim, rank, hidden):
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(12)
    part = MIXERS.get("wkv")({"hidden_size": hidden, "num_heads": heads, "head_dim": dim, "norm_eps": 1e-3}, env_for(k, dev, dtype))
    names = {f"mu_{s}": f"m.mu.{s}" for s in "rkvgw"}
    inner = heads * dim
    T = bind_part(part, g, dev, dtype, names, std=0.2, w1=[rank, hidden], w2=[inner, rank], w0=rnd(g, inner) - 1.5,
                  **{f"mu_{s}": torch.rand(hidden, generator=g, dtype=torch.float64) for s in "rkvgw"})
    h, h64 = lowered(rnd(g, 41, hidden), dtype, dev)
    head_close(run_part(part, h, dev, CUTS), plain.wkv_mixer(h64, T, "m", dict(heads=heads, dim=dim), 1e-3), tol * 2, dtype)
    with pytest.raises(ValueError):
        bind_part(part, g, dev, dtype, names, w1=[7, hidden], w2=[inner, 6])


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("left,right,hidden", [
    (dict(heads=4, kv_heads=2, dim=24, vdim=16, conv=3, mask={"size": 19}, scale=0.3, softcap=5.0, rot={"base": 100.0, "dims": 8}),
     dict(width=72, blocks=3, conv=4), 64),
    (dict(heads=2, kv_heads=1, dim=64, vdim=64, conv=1, scale=0.125, rot={"base": 5000.0, "dims": 64}), dict(width=64, blocks=1, conv=2), 128),
    (dict(heads=3, kv_heads=3, dim=10, vdim=14, conv=5, mask={"size": 8}, scale=0.4), dict(width=50, blocks=5, conv=1), 50)])
def test_the_two_mixers_side_by_side_are_the_plain_ones(backend, left, right, hidden):
    """The part as the plan builds it: one stacked input product, one state row for both, the inner norms."""
    k, dev, dtype, tol = setup(backend)
    g = torch.Generator().manual_seed(13)
    from simple_inference_amd.config import MeleraxConfig
    from simple_inference_amd.models.melerax import melerax_plan
    cfg = MeleraxConfig.from_dict({"architecture": "Melerax", "vocab": 8, "width": hidden, "norm": {"eps": 1e-3}, "layers": [
        {"type": "parallel", "mixer": {"left": left, "right": right}, "mlp": None}]})
    spec = melerax_plan(cfg).layers[0].parts["mixer"]
    part = MIXERS.get("parallel")(spec.params, env_for(k, dev, dtype))
    T = bind_part(part, g, dev, dtype, {local: name.replace("l0.mix", "m") for local, name in spec.weights.items()}, std=0.2)
    h, h64 = lowered(rnd(g, 41, hidden), dtype, dev)
    close(run_part(part, h, dev, CUTS), plain.side_by_side(h64, T, "m", {"left": left, "right": right}, 1e-3), tol * 2)


def test_what_does_not_combine_is_refused():
    from twins import TwinKernels
    env = env_for(TwinKernels(), "cpu", torch.float32)
    base = {"hidden_size": 32, "num_heads": 2, "num_kv_heads": 1, "head_dim": 16, "conv_taps": 2}
    for more in ({"value_from_key": True}, {"out_gate": True}, {"q_temp": {"coef": 1.0, "every": 2}}, {"value_mix": "gives"},
                 {"qk_norm": {"eps": 1e-5, "gain": False}}, {"conv_taps": 0}, {"qk_norm": {"eps": 1e-5, "over": "page"}}):
        with pytest.raises(ValueError):
            MIXERS.get("attention")({**base, **more}, env)
    unit = {"kind": "rglru", "params": {"hidden_size": 32, "width": 16, "blocks": 2, "conv_taps": 2}}
    with pytest.raises(ValueError):       # a norm behind one of two
        MIXERS.get("parallel")({"branches": {"a": {**unit, "norm": {"eps": 1e-5}}, "b": unit}}, env)
    with pytest.raises(ValueError):       # states that are not flat rows cannot share one
        gla = {"kind": "hgrn2", "params": {"hidden_size": 32, "num_heads": 2, "key_dim": 8, "value_dim": 8, "norm_eps": 1e-5}}
        MIXERS.get("parallel")({"branches": {"a": unit, "b": gla}}, env)
    with pytest.raises(ValueError):
        MIXERS.get("rglru")({"hidden_size": 32, "width": 16, "blocks": 3, "conv_taps": 2}, env)
