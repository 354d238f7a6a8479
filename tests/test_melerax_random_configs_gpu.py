"""Seeded random Melerax configurations through trace replay on the GPU, against the plain implementation: the three
mixers in any order and number, attention of any grouping of heads, widths of every kind and blocks from one position to
beyond the prompts, convolutions of one to six taps, linear units in any number of parts, matrix states with decay pairs of
any rank, dense and routed feed-forwards and none, tables of pairs of any size and none, widths and vocabularies that are
no multiple of anything.  Where a model errs more than the usual bound under bfloat16's rounding alone (the same replay with
the torch twins of the kernels, which round at the same places), the kernels may err up to twice that."""

import copy
import random

import pytest
import torch

import melerax_models as M
from test_trace_run import collect, make_trace

pytestmark = pytest.mark.gpu


def random_unit(rng):
    blocks = rng.choice([1, 2, 3, 8])
    return blocks * rng.choice([1, 5, 8, 16, 24, 40, 64, 80]), blocks, rng.choice([1, 2, 3, 4, 6])


def random_mixer(rng):
    kind = rng.choice(["parallel", "parallel", "wkv", "rglru"])
    if kind == "wkv":
        return M.wkv(rng.choice([1, 2, 3, 5]), rng.choice([8, 12, 16, 32, 40, 64, 96, 128]), rng.choice([1, 5, 8, 16, 24, 33, 64]))
    if kind == "rglru":
        return M.rglru(*random_unit(rng))
    kv, dim = rng.choice([1, 2, 3]), rng.choice([8, 10, 16, 20, 32, 48, 64, 96, 128, 160])
    turns = rng.random() < 0.8
    return M.parallel(M.attention(
        kv * rng.choice([1, 2, 4, 8]), kv, dim, rng.choice([8, 12, 16, 32, 64, 96, 128]), rng.choice([1, 2, 3, 4, 6]),
        rng.choice([None, 1, 2, 7, 16, 17, 30, 33, 64, 200]), rng.choice([0.05, 0.125, 0.3]), rng.choice([None, 1.0, 5.0, 30.0]),
        rng.choice([100.0, 10000.0, 250000.0]) if turns else None, rng.choice([d for d in (2, 4, 8, 16, dim) if d <= dim])),
        M.unit(*random_unit(rng)))


def random_mlp(rng):
    kind = rng.choice(["dense", "moe", "moe", None])
    if kind is None:
        return None
    sizes = [24, 30, 50, 64, 96, 136]
    if kind == "dense":
        return M.dense(rng.choice(sizes))
    count = rng.choice([1, 2, 4, 6])      # all are chosen: no close call between two experts decides a token
    return M.experts(count, count, rng.choice(sizes), rng.choice([None, *sizes]))


def random_config(seed):
    rng = random.Random(9000 + seed)
    shapes = [M.layer(random_mixer(rng), random_mlp(rng)) for _ in range(rng.choice([2, 3, 4]))]
    layers = [copy.deepcopy(rng.choice(shapes)) for _ in range(rng.choice([2, 3, 4, 5]))]
    vocab = rng.choice([97, 257, 500, 1001])
    return M.model(vocab, rng.choice([40, 72, 100, 128, 136, 192, 200, 264]), rng.choice([1e-5, 1e-6, 3e-4]),
                   rng.choice([None, (rng.choice([1, 7, 64, 509]), rng.choice([0, 1, 127, 1 << 20]), rng.choice([1, 17, 999983]))]),
                   layers)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(16))
def test_random_configuration_replays_like_the_plain_implementation(tmp_path, seed, dtype):
    from simple_inference_amd.replay import TraceReplayer

    cfg = random_config(seed)
    print("configuration", seed, cfg, flush=True)
    folder = M.write_model(tmp_path, cfg, seed=300 + seed, std=0.07, spread=0.3)
    steps, prompts, most = make_trace(cfg["vocab"], lengths=(50, 33, 71, 20, 64))
    page = (8, 16, 32, 64)[seed % 4]
    rp = TraceReplayer(folder, dtype, most, block_size=page, max_live=4)
    got = collect(steps, lambda st: rp.step(st["entries"], st["end"]).float().cpu().numpy())
    backend = "hip-f32" if dtype == "float32" else "hip-bf16"
    rounded = None
    if dtype == "bfloat16":     # what rounding at the same places costs this model, without this package's kernels
        from twins import TwinKernels
        twin = TraceReplayer(folder, dtype, most, block_size=page, max_live=4, device="cpu", kernels=TwinKernels())
        rounded = collect(steps, lambda st: twin.step(st["entries"], st["end"]).float().numpy())
    for r, toks in prompts.items():
        ref = M.plain_logits(folder, toks)
        mine = torch.stack([torch.as_tensor(got[r][p]) for p in range(len(toks))])
        bound = M.TOLERANCE[backend]
        if rounded is not None:
            theirs = torch.stack([torch.as_tensor(rounded[r][p]) for p in range(len(toks))])
            bound = max(bound, 2 * M.err(theirs, ref, backend))
        assert M.err(mine, ref, backend) <= bound, (r, M.err(mine, ref, backend), bound)
    assert all(rp.cache.free_pages(g) == -(-most // page) for g in range(len(rp.cache.groups))) and not rp.ids
    assert rp.cache.slots.free_slots == 4
