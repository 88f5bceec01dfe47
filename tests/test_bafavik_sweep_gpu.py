"""Random Bafavik configurations through the engine against the plain implementation: layer counts and orders of the three
mixers, feed-forwards or none, loops, token pairs or none, head counts in and out of the matrix cores' tiles, key, value, state
and width sizes, taps and ranks that differ from layer to layer, chunks of any size; three unequal requests side by side in
random portions with shuffled pages, and the longest alone."""
import random

import pytest
import torch

from bafavik_models import config, diff_att, draw_weights, heads, layer, parallel, parallel_2, rot, write_model
from helpers import engine_for, tolerance
from plain import bafavik_plain as P
from test_bafavik_gpu import run_schedule

pytestmark = pytest.mark.gpu


def random_heads(rng, rotated=True):
    h = rng.choice([1, 2, 3, 4, 6, 8, 16])
    kv = rng.choice([d for d in (1, 2, 3, 4, 8, 16) if h % d == 0])
    dim, vdim = rng.choice([8, 12, 16, 24, 32, 48, 64, 96, 128]), rng.choice([8, 16, 20, 32, 48, 64, 128, 256])
    dims = rng.choice([0, 2, dim // 2 // 2 * 2, dim]) if rotated else 0
    return h, kv, dim, vdim, rot(dims, rng.choice([50.0, 10000.0]))


def random_mixer(rng):
    kind = rng.choice(["attention", "parallel", "parallel", "parallel_2", "parallel_2"])
    h, kv, dim, vdim, turned = random_heads(rng, kind != "attention")
    if kind == "attention":
        return diff_att(h, kv, dim, vdim, chunk=rng.choice([None, 1, 3, 17, 33, 64, 65, 90, 400]), diff=rng.choice([0.0, 0.2, 0.7]))
    left = heads(h, kv, dim, vdim, **turned)
    h, kv, _, _, _ = random_heads(rng)
    dim, vdim = rng.choice([4, 8, 15, 16, 32, 48, 64, 96, 128]), rng.choice([8, 16, 20, 32, 48, 80])
    if kind == "parallel":
        return parallel(left, [rng.choice([0.2, 0.7, 0.95, 0.999, 1.0]) for _ in range(h)], dim, vdim, (rng.uniform(0.3, 1.5), rng.uniform(0.3, 1.5)))
    return parallel_2(left, rng.choice([1, 2, 3, 4, 5]), h, kv, dim, vdim, rng.choice([1, 2, 3, 4]))


def random_config(rng):
    layers = [layer(random_mixer(rng), rng.choice([None, 8, 40, 128, 128])) for _ in range(rng.randint(2, 5))]
    start = rng.randint(0, len(layers) - 1)
    loop = (start, rng.randint(start + 1, len(layers)), rng.choice([1, 2, 3])) if rng.random() < 0.6 else None
    bigram = (rng.choice([1, 7, 101]), rng.randint(1, 200), rng.randint(1, 200)) if rng.random() < 0.8 else None
    return config(rng.choice([48, 64, 96, 128, 256]), rng.choice([97, 256, 1000]), layers, eps=rng.choice([1e-4, 1e-5]),
                  scale=rng.choice([0.5, 1.0, 3.0]), bigram=bigram, mult=rng.choice([0.3, 1.0]), logit_scale=rng.choice([0.5, 1.0, 2.0]), loop=loop)


@pytest.mark.parametrize("seed", range(16))
def test_a_random_configuration_in_a_random_schedule(seed, tmp_path):
    rng = random.Random(7000 + seed)
    cfg = random_config(rng)
    ranks = {f"l{i}.mix.right.{s}": rng.choice([1, 5, 16, 64, 70]) for i in range(len(cfg["layers"])) for s in ("a1", "g1")}
    W = draw_weights(cfg, seed, ranks)
    folder = write_model(str(tmp_path / "model"), cfg, W)
    g = torch.Generator().manual_seed(seed)
    lengths = [rng.randint(1, 40), rng.randint(100, 300), rng.randint(40, 150)]
    seqs = {i: torch.randint(0, cfg["vocab"], (n,), generator=g).tolist() for i, n in enumerate(lengths)}
    Wd = {k: v.double() for k, v in W.items()}
    refs = {i: P.forward_logits(cfg, Wd, s).float() for i, s in seqs.items()}
    at, sched = {i: 0 for i in seqs}, []
    while any(at[i] < lengths[i] for i in seqs):
        step = []
        for i in seqs:
            if at[i] < lengths[i] and rng.random() < 0.8:
                n = min(rng.choice([1, 1, 2, 5, 16, 17, 33, 64, 100]), lengths[i] - at[i])
                step.append((i, n))
                at[i] += n
        if step:
            sched.append(step)
    for dtype in ("float32", "bfloat16"):
        eng = engine_for(folder, dtype, 64, 3 * 5 + 2, max_seqs=3, max_seq_len=320, shuffle_pages_seed=seed)
        got = run_schedule(eng, seqs, sched)
        got["alone"] = run_schedule(eng, {1: seqs[1]}, [[(1, lengths[1])]])[1]
        for i, rows in got.items():
            ref = refs[1 if i == "alone" else i]
            err = (rows - ref).abs().max(dim=-1).values / tolerance(dtype, ref)
            # a head's output is divided by its root mean square: a head that comes out small passes rounding on enlarged
            worst, middle = (8.0, 1.0) if dtype == "float32" else (12.0, 2.0)
            assert float(err.max()) <= worst and float(err.median()) <= middle, (i, dtype, float(err.max()), float(err.median()), cfg)
        eng.cache.check()
        assert not eng.live
