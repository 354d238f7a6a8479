"""The Melerax design through the engine's own step function, cache manager, state slots, scheduler and entry point,
against the plain implementation: every way of cutting the work must give the logits of the whole sequence.

The same tests run on the CPU with the torch twins of the kernels (they test configuration, plan, parts, cache
manager, state slots and batch layout) and on the GPU with the HIP kernels in float32 and bfloat16.
"""

import copy

import pytest
import torch

import melerax_models as M
from helpers import random_tokens
from test_mogisun_engine import cut, replay

BACKENDS = [
    pytest.param("twins"),
    pytest.param("twins-bf16"),
    pytest.param("hip-f32", marks=pytest.mark.gpu),
    pytest.param("hip-bf16", marks=pytest.mark.gpu),
]
FLOAT_BACKENDS = [pytest.param("twins"), pytest.param("hip-f32", marks=pytest.mark.gpu)]


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: M.write_model(tmp_path_factory.mktemp(f"melerax_{name}"), name, seed=5 + i)
            for i, name in enumerate(M.CONFIGS)}


def check(got, prompts, folder, backend):
    for req, rows in got.items():
        ref = M.plain_logits(folder, prompts[req])
        pos = sorted(rows)
        assert M.err(torch.stack([rows[p] for p in pos]), ref[pos], backend) <= M.TOLERANCE[backend], req


def test_configuration_reads_every_size_and_refuses_what_it_does_not_know():
    from simple_inference_amd.config import ConfigError, MeleraxConfig
    for name, cfg in M.CONFIGS.items():
        parsed = MeleraxConfig.from_dict(cfg)
        assert parsed.to_dict() == MeleraxConfig.from_dict(parsed.to_dict()).to_dict() == cfg
        assert parsed.vocab == cfg["vocab"] and parsed.width == cfg["width"] and len(parsed.layers) == len(cfg["layers"])
        assert parsed.norm_eps == cfg["norm"]["eps"]
    a = MeleraxConfig.from_dict(M.CONFIGS["a"])
    assert (a.bigram.buckets, a.bigram.mul_prev, a.bigram.mul_cur) == (61, 7, 5)
    left = a.layers[0].mixer.left
    assert (left.block, left.softcap, left.rot.dims, left.rot.base, left.conv, left.vdim) == (19, 5.0, 8, 10000.0, 3, 16)
    assert a.layers[3].mixer.left.softcap is None and a.layers[3].mlp is None and a.layers[5].mlp.shared_ff is None
    assert (a.layers[1].mlp.experts, a.layers[1].mlp.top, a.layers[1].mlp.ff, a.layers[1].mlp.shared_ff) == (5, 5, 24, 40)
    e = MeleraxConfig.from_dict(M.CONFIGS["e"])
    assert e.bigram is None and e.layers[3].mixer.left.block is None

    def broken(change):
        cfg = copy.deepcopy(M.CONFIGS["a"])
        change(cfg)
        with pytest.raises(ConfigError):
            MeleraxConfig.from_dict(cfg)
    broken(lambda c: c["layers"][1].update(type="gla"))
    broken(lambda c: c["layers"][0]["mlp"].update(kind="sparse"))
    broken(lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=3))
    broken(lambda c: c["layers"][0]["mixer"]["left"].pop("conv"))
    broken(lambda c: c["layers"][0]["mixer"]["left"].pop("scale"))
    broken(lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=26))
    broken(lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=7))
    broken(lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(scaling={"factor": 2.0, "original": 64, "fast": 8.0, "slow": 1.0}))
    broken(lambda c: c["layers"][0]["mixer"]["left"]["mask"].update(size=0))
    broken(lambda c: c["layers"][0]["mixer"]["left"].update(softcap=0))
    broken(lambda c: c["layers"][0]["mixer"].pop("right"))
    broken(lambda c: c["layers"][2]["mixer"].update(blocks=3))
    broken(lambda c: c["layers"][1]["mixer"].pop("heads"))
    broken(lambda c: c["layers"][1]["mlp"]["router"].update(top=6))
    broken(lambda c: c["layers"][1]["mlp"]["shared"].pop("ff"))
    broken(lambda c: c["embedding"]["bigram"].update(buckets=0))
    broken(lambda c: c["embedding"]["bigram"].update(mul_cur=-1))
    broken(lambda c: c.pop("width"))


def test_plan_gives_pages_and_states_to_whom_they_belong(folders):
    runner, cache = M.make_runner(folders["a"], "twins", 8, 16)
    layout = runner.model.cache_layout()
    assert layout.run_kv == [(0, 0), None, None, (1, 0), None, None] and layout.kv_slabs == [1, 1]
    first, second = layout.kv_groups
    assert (first.num_kv_heads, first.head_dim, first.value_dim, first.chunk) == (2, 24, 16, 19)
    assert (second.num_kv_heads, second.head_dim, second.value_dim, second.chunk) == (1, 12, 40, 33)
    assert layout.run_state == [0, 1, 2, 3, 4, 5] and layout.embedding_state == 6
    # the attention's ring of q, k and v channels, and behind it the unit's state with its own ring
    assert layout.states[0].shape == (3 * (4 * 24 + 2 * 24 + 2 * 16) + 72 * 5,)
    assert layout.states[1].shape == (3 * 16 * 16 + 96,)
    assert layout.states[2].shape == (80 * 3,)
    assert layout.states[6].shape == (1,) and layout.states[6].dtype == "int32"
    names = runner.model.expected_tensors()
    assert tuple(names["bigram"].shape) == (62, 96) and "l3.norm2" not in names and "l3.ls2" not in names
    assert names["l0.mix.left.q.norm"].shape == (96,) and names["l0.mix.left.k.norm"].shape == (48,)
    assert names["l0.mix.right.ra"].shape == (3, 24, 24) and "l5.mlp.shared.up" not in names
    assert M.make_runner(folders["e"], "twins", 8, 16)[0].model.cache_layout().embedding_state is None
    # one tap keeps nothing: a state for the unit alone, and none for the attention beside it
    one = M.make_runner(folders["b"], "twins", 8, 16)[0].model.cache_layout()
    assert one.states[0].shape == (64,) and one.states[1].shape == (32,)


def test_the_residual_after_every_layer_is_the_plain_one(folders):
    for name in ("a", "e"):
        runner, cache = M.make_runner(folders[name], "twins", 8, 16)
        toks = random_tokens(M.CONFIGS[name]["vocab"], 37, seed=3)
        cfg, w = M.read_model(folders[name])
        layers, _ = M.plain.layer_streams(cfg, w, toks)
        seen = []
        for built in runner.model.layers:
            original = built.block.forward

            def spy(stream, ctx, cache_, original=original):
                original(stream, ctx, cache_)
                seen.append(stream.residual.clone())
            built.block.forward = spy
        replay(runner, cache, [([(1, toks, [0])], [1])])
        assert len(seen) == len(cfg["layers"])
        for i, x in enumerate(seen):
            assert M.rel_err(x, layers[i]) < 2e-5, (name, i)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", list(M.CONFIGS))
def test_whole_prompt_then_token_by_token(folders, backend, name):
    folder = folders[name]
    runner, cache = M.make_runner(folder, backend, M.PAGE_SIZE[name], 40)
    toks = random_tokens(M.CONFIGS[name]["vocab"], 130, seed=7)
    n0 = 61        # the decoded tokens pass page borders and block edges
    schedule = [([(1, toks[:n0], list(range(n0)))], [])] + [([(1, [t], [0])], []) for t in toks[n0:]]
    got = replay(runner, cache, schedule)
    check(got, {1: toks}, folder, backend)
    # and all of it token by token, from the first token on
    cache.release(1)
    got = replay(runner, cache, [([(2, [t], [0])], []) for t in toks[:50]])
    check(got, {2: toks[:50]}, folder, backend)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name,sizes", [("a", [2, 5, 23, 1, 24, 3]), ("b", [19, 2, 2, 40, 1, 7]), ("c", [50, 17, 2, 33, 64]),
                                        ("e", [7, 2, 45, 1, 16]), ("f", [2, 2, 30, 3, 50])])
def test_portions_cut_anywhere_down_to_two_tokens(folders, backend, name, sizes):
    """Portions shorter than the convolutions' reach, portions that end in the middle of a page and of a block of
    positions: rings, states, the token before and the pages must carry over every cut."""
    folder = folders[name]
    runner, cache = M.make_runner(folder, backend, M.PAGE_SIZE[name], 40)
    toks = random_tokens(M.CONFIGS[name]["vocab"], 141, seed=8)
    got = replay(runner, cache, [([(1, part, list(range(len(part))))], []) for part in cut(toks, sizes)])
    check(got, {1: toks}, folder, backend)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["a", "c", "e"])
def test_unequal_requests_in_one_batch_with_pages_and_slots_used_again(folders, backend, name):
    """Up to three live requests of very different lengths: portions beside single tokens, requests left out of
    steps, requests that end and whose pages and state slots the next ones get.  The pool holds far less than all."""
    folder = folders[name]
    vocab = M.CONFIGS[name]["vocab"]
    lengths = [90, 7, 133, 41, 1, 66, 30]
    prompts = {i + 1: random_tokens(vocab, n, seed=100 + i) for i, n in enumerate(lengths)}
    plans = {r: cut(t[:-4], [11 + r, 2, 29]) + [[x] for x in t[-4:]] if len(t) > 4 else [[x] for x in t]
             for r, t in prompts.items()}
    waiting, live, schedule = list(prompts), [], []
    while waiting or live:
        while waiting and len(live) < 3:
            live.append(waiting.pop(0))
        entries, ends = [], []
        for r in list(live):
            if (len(schedule) + r) % 5 == 4 and len(live) > 1:
                continue
            part = plans[r].pop(0)
            entries.append((r, part, list(range(len(part)))))
            if not plans[r]:
                ends.append(r)
                live.remove(r)
        schedule.append((entries, ends))
    page = M.PAGE_SIZE[name]
    pool = sum(sorted(-(-n // page) for n in lengths)[-3:]) + 1
    runner, cache = M.make_runner(folder, backend, page, pool, max_running=3)
    got = replay(runner, cache, schedule)
    check(got, prompts, folder, backend)
    assert all(cache.free_pages(g) == pool for g in range(len(cache.groups))) and not cache.slots.slot_of
    # each alone gives the same (float32: to the last bits of the sums' order)
    if backend in ("twins", "hip-f32"):
        for r in (3, 6):
            solo = replay(runner, cache, [([(50 + r, prompts[r], list(range(len(prompts[r]))))], [50 + r])])
            for p, row in solo[50 + r].items():
                assert M.rel_err(row, got[r][p]) < 2e-5


@pytest.mark.parametrize("backend", BACKENDS)
def test_long_decoding(folders, backend):
    name = "c"
    folder = folders[name]
    runner, cache = M.make_runner(folder, backend, 16, 24)
    toks = random_tokens(300, 330, seed=9)
    wanted = {4, 5, 15, 16, 38, 39, 40, 41, 79, 80, 99, 100, 101, 150, 199, 200, 255, 256, 280, 299, 300, 329}
    schedule = [([(1, toks[:3], [0, 1, 2])], [])] + [([(1, [t], [0] if 3 + i in wanted else [])], [])
                                                    for i, t in enumerate(toks[3:])]
    got = replay(runner, cache, schedule)
    assert set(got[1]) == wanted | {0, 1, 2}
    check(got, {1: toks}, folder, backend)


def _long_memory(tensors):
    """Decays slowed down so that what was written hundreds of tokens back still weighs in the last logits."""
    for name, t in tensors.items():
        if name.endswith(".lam"):
            t.fill_(-9.0)
        elif name.endswith(".w0"):
            t.fill_(-7.0)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["c", "e"])
def test_a_far_token_reaches_the_last_logits_however_the_prompt_is_cut(folders, backend, tmp_path, name):
    """Two prompts that differ in one token hundreds of positions back: the last logits differ by far more than the
    tolerance, and by what the plain implementation says, in whole prompts, portions and decoding."""
    vocab = M.CONFIGS[name]["vocab"]
    folder = M.write_model(tmp_path / "far", name, seed=77, change=_long_memory)
    base = random_tokens(vocab, 420, seed=10)
    for place in (0, 16, 31):
        other = list(base)
        other[place] = (other[place] + 1) % vocab
        ref = [M.plain_logits(folder, p)[-1] for p in (base, other)]
        assert M.rel_err(ref[0], ref[1]) > 2e-4      # the far token matters: four times the float32 tolerance and more
        for sizes, tail in (([420], 0), ([37, 2, 161], 40)):
            rows = []
            for prompt in (base, other):
                runner, cache = M.make_runner(folder, backend, 16, 30)
                steps = [([(1, part, [])], []) for part in cut(prompt[:420 - tail - 1], sizes)]
                steps += [([(1, [t], [])], []) for t in prompt[420 - tail - 1:-1]] + [([(1, prompt[-1:], [0])], [])]
                rows.append(replay(runner, cache, steps)[1][419])
            for row, want in zip(rows, ref):
                assert M.err(row, want, backend) <= M.TOLERANCE[backend]
            if "bf16" not in backend:
                assert M.rel_err(rows[0], rows[1]) > 1e-4


@pytest.mark.parametrize("backend", FLOAT_BACKENDS)
@pytest.mark.parametrize("page", [8, 16])
def test_a_block_of_positions_sees_exactly_its_own_keys(backend, tmp_path, page):
    """A model of one layer whose linear unit's share is switched off, so that the last logits depend on the keys the last
    token sees (and on the tokens that the convolution of a visible key reaches) and on nothing else: they change if a
    token of the block changes, and stay the same to the last bit if it lies before what the block's first key
    reaches, in a whole prompt, in portions and in decoding; pages of finished blocks go back to the pool."""
    block, taps = 37, 3
    cfg = M.model(151, 64, 1e-5, None, [M.layer(M.parallel(
        M.attention(4, 2, 32, 32, taps, block, 0.3, 4.0, 3000.0, 16), M.unit(32, 2, 3)), M.dense(48))])

    def attention_only(tensors):
        tensors["l0.mix.right.out"].zero_()
    folder = M.write_model(tmp_path / "edge", cfg, seed=55, change=attention_only)
    for n in (150, 149, 148):       # the last token: third, second and first of its block
        start = (n - 1) // block * block
        base = random_tokens(151, n, seed=12)
        runs = (([n], 0), ([9, 2, 31], 30), ([2], n - 2))
        rows = {}

        def last(prompt, sizes, tail):
            runner, cache = M.make_runner(folder, backend, page, 30)
            steps = [([(1, part, [])], []) for part in cut(prompt[:n - tail - 1], sizes)]
            steps += [([(1, [t], [])], []) for t in prompt[n - tail - 1:-1]] + [([(1, prompt[-1:], [0])], [])]
            row = replay(runner, cache, steps)[1][n - 1]
            if tail > page:
                assert all(p < 0 for p in cache.table(0, 1)[:start // page])
            return row
        for i, (sizes, tail) in enumerate(runs):
            rows[i] = last(base, sizes, tail)
            assert M.rel_err(rows[i], M.plain_logits(folder, base)[-1]) < 5e-5
        for place, seen in ((start, True), (start - taps + 1, True), (start - taps, False), (start - 1, True), (0, False), (60, False)):
            other = list(base)
            other[place] = (other[place] + 1) % 151
            ref = M.plain_logits(folder, other)[-1]
            for i, (sizes, tail) in enumerate(runs):
                row = last(other, sizes, tail)
                assert M.rel_err(row, ref) < 5e-5
                assert torch.equal(row, rows[i]) != seen, (n, place, i)
                if seen:
                    assert M.rel_err(row, rows[i]) > 1e-4


@pytest.mark.parametrize("backend", FLOAT_BACKENDS)
@pytest.mark.parametrize("name", ["b", "e", "a"])
def test_a_state_slot_starts_from_zero_for_its_next_holder(folders, backend, name):
    """One slot: the second request gets the slot, the states, the rings and the last token that the first one left; its
    first tokens must not see them."""
    vocab = M.CONFIGS[name]["vocab"]
    runner, cache = M.make_runner(folders[name], backend, 16, 8, max_running=1)
    a, b = random_tokens(vocab, 40, seed=41), random_tokens(vocab, 25, seed=42)
    got = replay(runner, cache, [([(1, a, [39])], [1]), ([(2, b[:2], [0, 1])], []), ([(2, b[2:10], [0, 7])], []),
                                 ([(2, b[10:], [14])], [2])])
    check(got, {1: a, 2: b}, folders[name], backend)
    got = replay(runner, cache, [([(3, b[:1], [0])], []), ([(3, b[1:2], [0])], []), ([(3, b[2:3], [0])], [3])])
    check(got, {3: b}, folders[name], backend)
    assert cache.slots.free_slots == 1


@pytest.mark.parametrize("backend", FLOAT_BACKENDS)
def test_greedy_generation_through_the_engine_and_its_scheduler(folders, backend):
    from simple_inference_amd import Engine, EngineConfig, SamplingParams
    name = "c"
    if backend == "twins":
        from twins import TwinKernels
        kernels, device = TwinKernels(), "cpu"
    else:
        from simple_inference_amd.kernels import HipKernels
        kernels, device = HipKernels(), "cuda:0"
    eng = Engine.from_folder(folders[name], EngineConfig(
        device=device, dtype="float32", max_seq_len=128, block_size=16, max_running=3, chunk_tokens=24, eos_id=-1,
        num_kv_blocks=20), kernels)
    assert "Melerax" in eng.describe()
    prompts = [random_tokens(300, n, seed=300 + n) for n in (50, 3, 27, 85)]   # four requests for three slots
    reqs = [eng.add_request(p, params=SamplingParams(temperature=0.0, max_new_tokens=9)) for p in prompts]
    eng.run()
    cfg, w = M.read_model(folders[name])
    for req, prompt in zip(reqs, prompts):
        toks = list(prompt)
        assert len(req.generated) == 9
        for got in req.generated:
            logits = M.plain.forward(cfg, w, toks)[-1]
            want = int(torch.argmax(logits))
            assert got == want or float(logits[want] - logits[got]) < 1e-4 * float(logits.abs().max())
            toks.append(got)
    eng.cache.check()
    assert not eng.cache.lengths


def test_trace_replay_of_a_model_folder_on_the_cpu(folders):
    from simple_inference_amd.replay import TraceReplayer
    from twins import TwinKernels
    name = "a"
    rp = TraceReplayer(folders[name], "float32", 192, device="cpu", kernels=TwinKernels(), max_live=3)
    assert rp.describe().startswith("Melerax")
    a, b = random_tokens(211, 70, seed=31), random_tokens(211, 33, seed=32)
    out = rp.step([{"id": "x", "tokens": a[:40], "want": [39]}, {"id": "y", "tokens": b, "want": [0, 32]}], ["y"])
    out2 = rp.step([{"id": "x", "tokens": a[40:], "want": [29]}, {"id": "z", "tokens": b[:2], "want": [1]}], ["x", "z"])
    ra, rb = M.plain_logits(folders[name], a), M.plain_logits(folders[name], b)
    assert M.rel_err(out, torch.stack([ra[39], rb[0], rb[32]])) < 5e-5
    assert M.rel_err(out2, torch.stack([ra[69], rb[1]])) < 5e-5
    assert not rp.ids and rp.cache.free_pages() == 12 and rp.cache.slots.free_slots == 3


@pytest.mark.gpu
@pytest.mark.parametrize("name", ["a", "c"])
def test_bfloat16_generation_from_replayed_graphs_is_the_eager_one(folders, name):
    """The serving path: bfloat16, decode steps replayed from graphs, the host running ahead (the pairs' second token is
    then a sampled one that the host has not read).  The tokens are those of eager steps, and each is the plain
    implementation's best token or ties with it within bfloat16's reach."""
    from simple_inference_amd import Engine, EngineConfig, SamplingParams
    folder = folders[name]
    vocab = M.CONFIGS[name]["vocab"]
    prompts = [random_tokens(vocab, n, seed=400 + n) for n in (45, 70, 9)]
    runs = {}
    for graphs in (True, False):
        eng = Engine.from_folder(folder, EngineConfig(
            device="cuda:0", dtype="bfloat16", max_seq_len=256, block_size=16, max_running=4, chunk_tokens=64,
            eos_id=-1, use_graphs=graphs, run_ahead=graphs))
        reqs = [eng.add_request(p, params=SamplingParams(temperature=0.0, max_new_tokens=40)) for p in prompts]
        eng.run()
        runs[graphs] = [list(r.generated) for r in reqs]
        if graphs:
            assert eng.graphs is not None and eng.stats["graph_fallbacks"] == 0
    assert runs[True] == runs[False]
    cfg, w = M.read_model(folder)
    for prompt, generated in zip(prompts, runs[True]):
        toks = list(prompt)
        for got in generated:
            logits = M.plain.forward(cfg, w, toks)[-1]
            want = int(torch.argmax(logits))
            assert got == want or float(logits[want] - logits[got]) < 5e-2 * float(logits.abs().max())
            toks.append(got)
