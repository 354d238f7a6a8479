"""The Lunerax design through the engine's own step function, cache manager, state slots, scheduler and entry point,
against the plain implementation: every way of cutting the work must give the logits of the whole sequence.

The same tests run on the CPU with the torch twins of the kernels (they test configuration, plan, parts, cache
manager, state slots and batch layout) and on the GPU with the HIP kernels in float32 and bfloat16.
"""

import copy

import pytest
import torch

import lunerax_models as M
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
    return {name: M.write_model(tmp_path_factory.mktemp(f"lunerax_{name}"), name, seed=5 + i)
            for i, name in enumerate(M.CONFIGS)}


def check(got, prompts, folder, backend):
    for req, rows in got.items():
        ref = M.plain_logits(folder, prompts[req])
        pos = sorted(rows)
        assert M.err(torch.stack([rows[p] for p in pos]), ref[pos], backend) <= M.TOLERANCE[backend], req


def test_configuration_reads_every_size_and_refuses_what_it_does_not_know():
    from simple_inference_amd.config import ConfigError, LuneraxConfig
    for name, cfg in M.CONFIGS.items():
        parsed = LuneraxConfig.from_dict(cfg)
        assert parsed.to_dict() == LuneraxConfig.from_dict(parsed.to_dict()).to_dict() == cfg
        assert parsed.vocab == cfg["vocab"] and parsed.width == cfg["width"] and len(parsed.layers) == len(cfg["layers"])
        assert parsed.embedding_scale == cfg["embedding"]["scale"] and parsed.norm_eps == cfg["norm"]["eps"]
        assert parsed.logit_softcap == cfg.get("logit_softcap")
        assert parsed.side_dim == (cfg["token_side"]["dim"] if "token_side" in cfg else None)
    a = LuneraxConfig.from_dict(M.CONFIGS["a"])
    assert (a.layers[0].mixer.window, a.layers[0].mixer.keep_first, a.layers[0].mixer.softcap) == (11, 3, 5.0)
    assert a.layers[3].mixer.softcap is None and a.layers[3].mlp is None and not a.layers[3].mixer.v_mix
    assert a.layers[2].mixer.window == 13 and a.layers[2].mixer.rot.base == 10000.0
    assert LuneraxConfig.from_dict(M.CONFIGS["e"]).layers[3].mixer.window is None

    def broken(change):
        cfg = copy.deepcopy(M.CONFIGS["a"])
        change(cfg)
        with pytest.raises(ConfigError):
            LuneraxConfig.from_dict(cfg)
    broken(lambda c: c["layers"][1].update(type="delta"))
    broken(lambda c: c["layers"][0]["mlp"].update(kind="moe"))
    broken(lambda c: c["layers"][1]["mixer"].update(kv_heads=3))
    broken(lambda c: c["layers"][1]["mixer"].pop("conv"))
    broken(lambda c: c["layers"][2]["mixer"].pop("q_rank"))
    broken(lambda c: c["layers"][2]["mixer"]["rot"].update(dims=18))
    broken(lambda c: c["layers"][2]["mixer"]["rot"].update(scaling={"factor": 2.0, "original": 64, "fast": 8.0, "slow": 1.0}))
    broken(lambda c: c["layers"][2]["mixer"]["mask"].update(keep_first=2))
    broken(lambda c: c["layers"][0]["mixer"]["mask"].update(keep_first=-1))
    broken(lambda c: c["layers"][0]["mixer"]["mask"].pop("size"))
    broken(lambda c: c["layers"][0]["mixer"].update(softcap=0))
    broken(lambda c: c["layers"][0]["mixer"].update(v_mix=1))
    broken(lambda c: c["layers"][5]["mixer"].update(vdim=20))      # mixes with layer 0's values of width 16
    broken(lambda c: c["token_side"].update(dim=0))
    broken(lambda c: c.pop("width"))


def test_plan_gives_pages_and_states_to_whom_they_belong(folders):
    runner, cache = M.make_runner(folders["a"], "twins", 8, 16)
    layout = runner.model.cache_layout()
    assert layout.run_kv == [(0, 0), None, (1, 0), (2, 0), None, (3, 0)] and layout.kv_slabs == [1, 1, 1, 1]
    first, second, third, fourth = layout.kv_groups
    assert (first.num_kv_heads, first.head_dim, first.value_dim, first.window, first.keep_first) == (2, 24, 16, 11, 3)
    assert (second.num_kv_heads, second.head_dim, second.value_dim, second.window) == (1, 48, 40, 13)
    assert third.keep_first == 12 and fourth.keep_first == 0
    assert layout.run_state == [None, 0, None, None, 1, None]
    # the matrices, and behind them the convolution's kept inputs: (taps - 1) rows of q, k and v channels
    assert layout.states[0].shape == (4 * 12 * 20 + (2 * 2 * 12 + 4 * 20) * 3,)
    assert layout.states[1].shape == (3 * 16 * 8 + (2 * 3 * 16 + 3 * 8) * 1,)
    mixing = [getattr(part.mixer, "value_mix", None) for part in runner.model.layers]
    assert mixing == ["gives", None, None, None, None, "takes"]
    names = runner.model.expected_tensors()
    assert tuple(names["side.embed"].shape) == (211, 6 * 20) and "l3.norm2" not in names and "l0.mix.vmix" in names
    assert "l3.mix.vmix" not in names and names["l2.mix.g"].shape == (72, 96) and names["final.norm.b"].shape == (96,)
    assert "side.embed" not in M.make_runner(folders["f"], "twins", 8, 16)[0].model.expected_tensors()


def test_the_residual_after_every_layer_is_the_plain_one(folders):
    """Layer by layer: what is pending after a block is settled into a copy of its residual."""
    from simple_inference_amd.parts.context import ResidualStream
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
                probe = ResidualStream(stream.residual.clone(), stream.raw_delta)
                probe.post = stream.post
                seen.append(probe.settle(ctx.kernels).clone())
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
    n0 = 61        # the decoded tokens pass page borders and every window
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
    """Portions shorter than the convolution's reach and than the windows, portions that end in the middle of a page and
    among the kept first tokens: the convolution's kept inputs, the states and the pages must carry over every cut."""
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
    wanted = {4, 5, 6, 15, 16, 19, 20, 21, 44, 45, 46, 74, 75, 76, 89, 90, 91, 150, 200, 255, 256, 299, 300, 329}
    schedule = [([(1, toks[:3], [0, 1, 2])], [])] + [([(1, [t], [0] if 3 + i in wanted else [])], [])
                                                    for i, t in enumerate(toks[3:])]
    got = replay(runner, cache, schedule)
    assert set(got[1]) == wanted | {0, 1, 2}
    check(got, {1: toks}, folder, backend)


def _long_memory(tensors):
    """Decays slowed down so that what was written hundreds of tokens back still weighs in the last logits."""
    for name, t in tensors.items():
        if name.endswith(".mix.A_log"):
            t.fill_(-6.0)


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


ONE_LAYER = {
    "capped": (M.model(151, 64, 1e-5, 2.0, 12, 9.0, [M.layer(M.attention(4, 2, 32, 32, 21, 3, 0.3, 4.0, True), 48)]), 21, 3),
    # more kept tokens than a page holds, and than the window
    "kept": (M.model(151, 64, 1e-5, 2.0, 12, None, [M.layer(M.attention(2, 2, 16, 24, 9, 19, 0.3, None, False), None)]), 9, 19),
    "latent": (M.model(151, 64, 1e-5, 2.0, None, 9.0, [M.layer(M.latent(3, 16, 8, 24, 32, 40, 27, 0.3, 3000.0), 48)]), 27, 0),
}


@pytest.mark.parametrize("backend", FLOAT_BACKENDS)
@pytest.mark.parametrize("which", list(ONE_LAYER))
@pytest.mark.parametrize("page", [8, 16])
def test_a_window_sees_exactly_its_keys_and_the_kept_first_ones(backend, tmp_path, which, page):
    """A model of one layer, whose last logits depend on the keys the last token sees and on nothing else: they change if
    a token just inside the window or among the kept first ones changes, and stay the same to the last bit if it is one
    further out, in a whole prompt, in portions and in decoding; pages behind the window go back to the pool, those of
    the first tokens do not."""
    cfg, window, keep = ONE_LAYER[which]
    folder = M.write_model(tmp_path / "edge", cfg, seed=55)
    n = 150
    base = random_tokens(151, n, seed=12)
    places = [(n - window, True), (n - window - 1, False), (keep, False), (60, False)] + ([(keep - 1, True), (0, True)] if keep else [(0, False)])
    runs = (([n], 0), ([9, 2, 31], 30), ([2], n - 2))
    rows = {}

    def last(prompt, sizes, tail):
        runner, cache = M.make_runner(folder, backend, page, 30)
        steps = [([(1, part, [])], []) for part in cut(prompt[:n - tail - 1], sizes)]
        steps += [([(1, [t], [])], []) for t in prompt[n - tail - 1:-1]] + [([(1, prompt[-1:], [0])], [])]
        row = replay(runner, cache, steps)[1][n - 1]
        table = cache.table(0, 1)
        kept = -(-keep // page)
        assert all(p >= 0 for p in table[:kept])
        held = len([p for p in table if p >= 0])
        assert held <= -(-(window + max(sizes)) // page) + 1 + kept
        if tail > window + page:        # long after the last portion only the window's pages are left
            assert all(p < 0 for p in table[kept:(n - window) // page])
        return row
    for i, (sizes, tail) in enumerate(runs):
        rows[i] = last(base, sizes, tail)
        assert M.rel_err(rows[i], M.plain_logits(folder, base)[-1]) < 5e-5
    for place, seen in places:
        other = list(base)
        other[place] = (other[place] + 1) % 151
        ref = M.plain_logits(folder, other)[-1]
        for i, (sizes, tail) in enumerate(runs):
            row = last(other, sizes, tail)
            assert M.rel_err(row, ref) < 5e-5
            assert torch.equal(row, rows[i]) != seen, (place, i)
            if seen:
                assert M.rel_err(row, rows[i]) > 1e-4


@pytest.mark.parametrize("backend", FLOAT_BACKENDS)
@pytest.mark.parametrize("name", ["b", "e"])
def test_a_state_slot_starts_from_zero_for_its_next_holder(folders, backend, name):
    """One slot: the second request gets the slot, the matrices and the convolution's kept inputs that the first one
    left; its first tokens, which the convolution pads with zeros, must not see them."""
    vocab = M.CONFIGS[name]["vocab"]
    runner, cache = M.make_runner(folders[name], backend, 16, 8, max_running=1)
    a, b = random_tokens(vocab, 40, seed=41), random_tokens(vocab, 25, seed=42)
    got = replay(runner, cache, [([(1, a, [39])], [1]), ([(2, b[:2], [0, 1])], []), ([(2, b[2:10], [0, 7])], []),
                                 ([(2, b[10:], [14])], [2])])
    check(got, {1: a, 2: b}, folders[name], backend)
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
    assert "Lunerax" in eng.describe()
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
    assert rp.describe().startswith("Lunerax")
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
    """The serving path: bfloat16, decode steps replayed from graphs, the host running ahead.  The tokens are those
    of eager steps, and each is the plain implementation's best token or ties with it within bfloat16's reach."""
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
