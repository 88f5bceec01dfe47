"""Random Lilunex configurations through the engine against the plain implementation: layer counts and orders of the
three mixers, feed-forwards dense, routed (with and without identities and a shared expert) or none, head counts in and
out of the matrix cores' tiles, key, value, state and width sizes that differ from layer to layer, windows and kept
positions of any size, layers that read an earlier layer's keys under a mask of their own; three unequal requests side
by side in random portions with shuffled pages, and the longest alone."""
import random

import pytest
import torch

from helpers import engine_for, tolerance
from lilunex_models import att, config, delta, dense, draw_weights, layer, moe, wkv, write_model
from plain import lilunex_plain as P
from test_lilunex_gpu import SLACK, run_schedule

pytestmark = pytest.mark.gpu


def random_mask(rng):
    return rng.choice([None, (rng.choice([1, 3, 17, 33, 64, 65, 90, 400]), rng.choice([0, 1, 4, 16, 64, 70])),
                       (rng.randint(1, 200), rng.randint(0, 12))])


def random_layer(rng, layers):
    kind = rng.choice(["wkv", "attention", "attention", "delta"])
    if kind == "wkv":
        return wkv(rng.choice([1, 2, 3, 4, 8]), rng.choice([4, 8, 15, 16, 32, 64, 96]))
    heads = rng.choice([1, 2, 3, 4, 6, 8, 16])
    kv_heads = rng.choice([d for d in (1, 2, 3, 4, 8, 16) if heads % d == 0])
    dim, vdim = rng.choice([8, 12, 16, 24, 32, 48, 64, 96, 128]), rng.choice([8, 16, 20, 32, 48, 64, 96])
    if kind == "delta":
        return delta(heads, kv_heads, dim, vdim, rng.choice([1, 2, 3, 4]))
    own = [i for i, L in enumerate(layers) if L["type"] == "attention" and L["mixer"].get("kv_from") is None]
    if own and rng.random() < 0.5:
        j = rng.choice(own)
        m = layers[j]["mixer"]
        return {"type": "attention", "mixer": {**{k: v for k, v in m.items() if k != "mask"}, "kv_from": j,
                                               **({"mask": {"size": mask[0], "keep_first": mask[1]}} if (mask := random_mask(rng)) else {})}}
    dims = rng.choice([0, 2, dim // 2 // 2 * 2, dim])
    rot = (dims, rng.choice([50.0, 10000.0]), rng.choice([None, 2.0, 8.0])) if dims else None
    return att(heads, kv_heads, dim, vdim, mask=random_mask(rng), rot=rot)


def random_config(rng):
    layers = []
    for _ in range(rng.randint(2, 6)):
        mlp, pick = None, rng.random()
        if pick < 0.4:
            mlp = dense(rng.choice([8, 40, 128]))
        elif pick < 0.85:
            experts, identity = rng.choice([1, 2, 4, 5, 8, 16]), rng.choice([0, 1, 4])
            mlp = moe(experts, identity, rng.randint(1, min(experts + identity, 4)), rng.choice([8, 24, 64]), rng.choice([None, 16, 96]))
        layers.append(layer(random_layer(rng, layers), mlp))
    return config(rng.choice([48, 64, 96, 128, 256]), rng.choice([97, 256, 1000]), layers, eps=rng.choice([1e-4, 1e-5]),
                  scale=rng.choice([0.5, 1.0, 3.0]))


@pytest.mark.parametrize("seed", range(16))
def test_a_random_configuration_in_a_random_schedule(seed, tmp_path):
    rng = random.Random(5000 + seed)
    cfg = random_config(rng)
    W = draw_weights(cfg, seed, {i: rng.choice([1, 5, 16, 64, 70]) for i in range(len(cfg["layers"]))})
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
        got, chose = run_schedule(eng, cfg, seqs, sched)
        alone, chose_alone = run_schedule(eng, cfg, {1: seqs[1]}, [[(1, lengths[1])]])
        got["alone"], chose["alone"] = alone[1], chose_alone[1]
        for i, rows in got.items():
            r = 1 if i == "alone" else i
            # 16 bits: the plain run takes the engine's experts where these are a close call of its own choice
            ref = refs[r] if dtype == "float32" else P.forward_logits(cfg, Wd, seqs[r], chose[i], SLACK).float()
            err = (rows - ref).abs().max(dim=-1).values / tolerance(dtype, ref)
            if dtype == "float32":
                # a head's output is divided by its root mean square: a head that comes out small passes rounding on enlarged
                assert float(err.max()) <= 8.0 and float(err.median()) <= 1.0, (i, float(err.max()), float(err.median()), cfg)
            else:
                assert float(err.max()) <= 12.0 and float(err.median()) <= 2.0, (i, float(err.max()), float(err.median()), cfg)
        eng.cache.check()
        assert not eng.live
