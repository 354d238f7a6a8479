"""Seeded random Lunerax configurations through trace replay on the GPU, against the plain implementation: the three
mixers in any order and number, delta rules with any grouping of heads, widths of every kind, convolutions of one to
five taps and low-rank pairs of any rank, latent attention with and without a window, capped attention with windows from
one token to beyond the prompts, none to many kept first tokens, with and without a cap and mixed values, layers without
a feed-forward, second embeddings of any width or none, widths and vocabularies that are no multiple of anything.  Where
a model errs more than the usual bound under bfloat16's rounding alone (the same replay with the torch twins of the
kernels, which round at the same places), the kernels may err up to twice that."""

import copy
import random

import pytest
import torch

import lunerax_models as M
from test_trace_run import collect, make_trace

pytestmark = pytest.mark.gpu


def random_mixer(rng, value_heads):
    kind = rng.choice(["delta", "latent", "attention"])
    kv = rng.choice([1, 2, 3])
    if kind == "delta":
        return M.delta(kv * rng.choice([1, 2, 4]), kv, rng.choice([8, 20, 32, 48, 64, 128]), rng.choice([8, 12, 32, 64, 80, 128]),
                       rng.choice([1, 2, 3, 4, 5]), rng.choice([1, 7, 8, 24, 40, 64]), rng.choice([3, 8, 16, 33]))
    window = rng.choice([None, 1, 2, 7, 16, 17, 31, 40, 64, 200])
    if kind == "latent":
        rot = rng.choice([2, 6, 8, 16, 32, 64])
        return M.latent(rng.choice([1, 2, 3, 5, 8, 17]), rng.choice([8, 12, 32, 64]), rot, rng.choice([8, 20, 32, 64]),
                        rng.choice([16, 20, 64, 96]), rng.choice([16, 24, 40, 96, 128, 264]), window, rng.choice([0.05, 0.125, 0.3]),
                        rng.choice([100.0, 10000.0, 250000.0]), rng.choice([d for d in (2, 4, 8, 16, rot) if d <= rot]))
    mix = rng.random() < 0.6
    if mix:
        kv, vdim = value_heads
    else:
        vdim = rng.choice([8, 12, 32, 64, 128])
    return M.attention(kv * rng.choice([1, 2, 4]), kv, rng.choice([8, 20, 32, 64, 96, 128, 160]), vdim, window,
                       rng.choice([0, 1, 3, 8, 17, 40]) if window else 0, rng.choice([0.05, 0.125, 0.3]),
                       rng.choice([None, 1.0, 5.0, 30.0]), mix)


def random_config(seed):
    rng = random.Random(8000 + seed)
    value_heads = (rng.choice([1, 2, 3]), rng.choice([8, 20, 32, 64]))
    shapes = [M.layer(random_mixer(rng, value_heads), rng.choice([None, 24, 50, 64, 136, 256])) for _ in range(rng.choice([2, 3, 4]))]
    layers = [copy.deepcopy(rng.choice(shapes)) for _ in range(rng.choice([2, 3, 4, 5, 6]))]
    return M.model(rng.choice([97, 257, 500, 1001]), rng.choice([40, 72, 100, 128, 136, 192, 200, 264]), rng.choice([1e-5, 1e-6, 3e-4]),
                   rng.choice([1.0, 3.0, 12.0]), rng.choice([None, 3, 16, 64, 72]), rng.choice([None, 4.0, 25.0]), layers)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(14))
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
