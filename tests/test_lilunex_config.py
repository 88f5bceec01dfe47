"""Lilunex configurations as data, the sizes that only tensors tell, refusals, caches that keep what their readers
need, and the plain implementation's pieces pinned against library routines."""
import copy
import math

import pytest
import torch

from axon_amd.cache import CacheManager, GroupPlan
from axon_amd.config import ConfigError, LilunexConfig, config_from_dict
from axon_amd.engine.loading import read_model_config
from axon_amd.models import build_model_description
from axon_amd.parts import CacheSpec
from axon_amd.weights import Checkpoint, CheckpointSource, WeightError, check_tensors, write_random_model
from lilunex_models import MODELS, draw_weights, make
from plain import lilunex_plain as P


@pytest.mark.parametrize("name", sorted(MODELS))
def test_a_checkpoint_fits_what_the_parts_declare(name, tmp_path):
    folder = make(str(tmp_path), name)
    ck = Checkpoint(folder)
    cfg = read_model_config(folder, ck)
    assert isinstance(cfg, LilunexConfig) and cfg.to_dict() == MODELS[name]["cfg"]
    model = build_model_description(cfg)
    check_tensors(model.tensors(), CheckpointSource(ck), cfg.ignores_tensor)
    # the ranks come from the tensors' shapes
    for i, rank in MODELS[name]["rank"].items():
        assert model.blocks[i].mixer.rank == rank
    assert [r.layer for r in model.order] == list(range(len(cfg.layers)))


def test_constants_of_the_configuration_reach_the_parts():
    spec = config_from_dict(MODELS["A"]["cfg"]).model_spec()
    a, b = spec.layers[1].mixer.params, spec.layers[3].mixer.params
    assert a["mask"] == {"kind": "window", "size": 7, "keep": 3} and b["mask"] == {"kind": "window", "size": 12, "keep": 9}
    assert a["position"].params["scaling"] == {"kind": "linear", "factor": 2.0} and a["position"].params["rotary_dim"] == 4
    assert not a["reads_cache"] and b["reads_cache"] and a["qk_norm"] == "rows" and a["sink"] == "heads"
    assert [(r.cache, r.writes_cache) for r in spec.order] == [(0, True), (1, True), (2, True), (1, False), (4, True)]
    ff = spec.layers[1].feed_forward.params
    assert (ff["experts"], ff["identity"], ff["top"], ff["ff"]) == (5, 2, 2, 24) and ff["shared"] == {"ff": 16, "unit": "gated", "gate": "sg"}
    assert spec.layers[0].feed_forward.params["activation"] == "relu_squared" and spec.layers[2].feed_forward is None
    assert spec.embedding.params["scale"] == 1.5 and spec.layers[0].mixer.params["eps"] == 1e-5


def test_a_cache_keeps_what_any_of_its_readers_sees():
    plan = lambda name: build_model_description(config_from_dict(MODELS[name]["cfg"])).cache_plan
    # A: layer 1 (window 7, 3 kept) and its reader (12, 9)
    (spec,) = plan("A").group_specs
    assert (spec.window, spec.keep) == (12, 9)
    # B: (70, 4) and its reader (130, 0); (40, 66) and its reader (9, 2)
    assert sorted((s.window, s.keep) for s in plan("B").group_specs) == [(40, 66), (130, 4)]
    # D: a reader without a mask needs every position
    assert [(s.window, s.keep) for s in plan("D").group_specs] == [(0, 0), (0, 0)]
    assert plan("E").group_specs == [] and len(plan("E").state_elems) == 3
    bindings = plan("B").bindings
    assert (bindings[4].group, bindings[4].index, bindings[4].writes) == (bindings[0].group, bindings[0].index, False)


def test_random_weights_round_trip(tmp_path):
    cfg = config_from_dict(MODELS["B"]["cfg"])
    folder = write_random_model(cfg, str(tmp_path / "m"), seed=3)
    back = read_model_config(folder)
    check_tensors(build_model_description(back).tensors(), CheckpointSource(Checkpoint(folder)))
    assert back.layers[2]["mixer"].params["rank"] == cfg.layers[2]["mixer"].params["rank"] == 16


@pytest.mark.parametrize("edit,fragment", [
    (lambda c: c["layers"][3]["mixer"].update(kv_from=4), "not an attention layer before it"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=0), "not an attention layer before it"),
    (lambda c: c["layers"][3]["mixer"].update(dim=12), "its dim 10 is not this layer's 12"),
    (lambda c: c["layers"][0].update(type="rglru"), "is not a mixer of this design"),
    (lambda c: c["layers"][0]["mlp"].update(kind="glu"), "is not a feed-forward of this design"),
    (lambda c: c["layers"][1]["mixer"].update(heads=3), "not a multiple of"),
    (lambda c: c["layers"][1]["mixer"]["mask"].update(size=0), "at least 1"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=8), "experts a token"),
    (lambda c: c["layers"][2]["mixer"].update(dim=300), "takes 1 to 256"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=3), "must be even"),
    (lambda c: c.update(layers=[]), "not a list of layers"),
    (lambda c: c.pop("norm"), "is not an object"),
])
def test_refusals(edit, fragment):
    cfg = copy.deepcopy(MODELS["A"]["cfg"])
    edit(cfg)
    with pytest.raises(ConfigError, match=fragment):
        build_model_description(config_from_dict(cfg))


def test_a_missing_low_rank_matrix_is_reported_with_the_rest(tmp_path):
    from lilunex_models import write_model
    m = MODELS["E"]
    W = draw_weights(m["cfg"], 1, m["rank"])
    del W["l0.mix.w1"], W["l1.mix.q.conv"]
    folder = write_model(str(tmp_path), m["cfg"], W)
    cfg = read_model_config(folder)
    with pytest.raises(WeightError) as e:
        check_tensors(build_model_description(cfg).tensors(), CheckpointSource(Checkpoint(folder)))
    assert {"l0.mix.w1", "l1.mix.q.conv"} <= set(e.value.missing)


# --------------------------------------------------------------------------- pages under a window beside kept positions
def test_a_window_never_gives_back_the_pages_of_kept_positions():
    cm = CacheManager([GroupPlan(CacheSpec(1, 1, 8, 20, keep=9), 1, 8, 12), GroupPlan(CacheSpec(1, 1, 4, 20), 1, 8, 12)], [], 2, 256)
    s = cm.open()
    for n in range(1, 121):
        cm.reserve(s, n)
        cm.trim(s, n)
        lo = max(0, n + 1 - 20) // 8                    # the first page the window of the next token touches
        held = -(-n // 8)
        assert cm.pages_of(0, s) == held - max(0, lo - 2) and cm.pages_of(1, s) == held - min(lo, held)
        row = cm.row(0, s)
        if n > 60:
            assert len(set(row[:2])) == 2 and all(row[i] == 0 for i in range(2, lo))
        cm.check()
    assert cm.close(s) > 0 and cm.free_pages(0) == cm.free_pages(1) == 12


# --------------------------------------------------------------------------- pins of the plain implementation
def test_the_plain_attention_is_a_library_attention_without_sink_and_window():
    g = torch.Generator().manual_seed(1)
    q, k, v = (torch.randn(9, n, 6, generator=g, dtype=torch.float64) for n in (4, 2, 2))
    none = torch.full((4,), -1e9, dtype=torch.float64)
    got = P.heads_attention(q, k, v, 0.3, None, none)
    rep = lambda x: x.repeat_interleave(2, dim=1).transpose(0, 1)
    want = torch.nn.functional.scaled_dot_product_attention(q.transpose(0, 1), rep(k), rep(v), is_causal=True, scale=0.3).transpose(0, 1)
    assert torch.allclose(got, want, atol=1e-12)
    # a sink is a key whose value is zero
    sink = torch.tensor([0.5, -1.0, 2.0, 0.0], dtype=torch.float64)
    got = P.heads_attention(q, k, v, 0.3, {"size": 3, "keep_first": 1}, sink)
    for a in range(4):
        for i in range(9):
            js = [j for j in range(i + 1) if i - j < 3 or j < 1]
            s = torch.cat([(k[js, a // 2] @ q[i, a]) * 0.3, sink[a][None]])
            assert torch.allclose(got[i, a], torch.softmax(s, 0)[:-1] @ v[js, a // 2], atol=1e-12)


def test_the_plain_recurrences_reduce_to_sums():
    g = torch.Generator().manual_seed(2)
    r, k, v = (torch.randn(7, 2, 4, generator=g, dtype=torch.float64) for _ in range(3))
    w = torch.rand(7, 2, 4, generator=g, dtype=torch.float64)
    u = torch.randn(2, 4, generator=g, dtype=torch.float64)
    got = P.wkv_recurrence(r, k, v, w, u)
    for t in range(7):
        want = (r[t] * u * k[t]).sum(-1, keepdim=True) * v[t]
        for s in range(t):
            carried = torch.prod(w[s + 1:t], dim=0)
            want = want + (r[t] * carried * k[s]).sum(-1, keepdim=True) * v[s]
        assert torch.allclose(got[t], want, atol=1e-12)
    # the delta rule on orthonormal keys without decay and with beta 1 stores what it is given, and a key met again
    # replaces its value
    eye = torch.eye(4, dtype=torch.float64)
    keys = eye[[0, 1, 2, 0]][:, None, :]
    vals = torch.randn(4, 1, 3, generator=g, dtype=torch.float64)
    one = torch.ones(4, 1, dtype=torch.float64)
    out = P.delta_recurrence(keys, keys, vals, one, one)
    assert torch.allclose(out, vals, atol=1e-12)
    reads = P.delta_recurrence(eye[[3, 3, 3, 1]][:, None, :], keys, vals, one, one)
    assert torch.allclose(reads[3], vals[1], atol=1e-12) and float(reads[:3].abs().max()) == 0.0


def test_the_plain_rotation_is_a_complex_product_and_the_norms_library_ones():
    g = torch.Generator().manual_seed(3)
    v = torch.randn(5, 2, 10, generator=g, dtype=torch.float64)
    pos = torch.tensor([0, 1, 7, 100, 4000])
    got = P.rotate_halves(v, pos, {"dims": 6, "base": 50.0, "scaling": {"factor": 4.0}})
    z = torch.complex(v[..., :3], v[..., 3:6])
    turn = torch.exp(1j * pos[:, None].double() * (50.0 ** (-2.0 * torch.arange(3).double() / 6) / 4.0))
    z = z * turn[:, None, :]
    assert torch.allclose(got, torch.cat([z.real, z.imag, v[..., 6:]], -1), atol=1e-12)
    x = torch.randn(3, 8, generator=g, dtype=torch.float64)
    assert torch.allclose(P.unit(x, 0.1), torch.nn.functional.rms_norm(x, (8,), eps=0.1), atol=1e-12)
    assert torch.allclose(P.softplus(x), torch.nn.functional.softplus(x), atol=1e-9)
    assert torch.allclose(P.silu(x), torch.nn.functional.silu(x), atol=1e-12)


def test_a_correction_chooses_and_does_not_weigh():
    W = {"router": torch.eye(3, dtype=torch.float64), "correction": torch.tensor([0.0, 0.9, 0.0], dtype=torch.float64)}
    for e in range(2):
        W.update({f"e{e}.gate": torch.zeros(1, 3, dtype=torch.float64), f"e{e}.up": torch.zeros(1, 3, dtype=torch.float64),
                  f"e{e}.down": torch.zeros(3, 1, dtype=torch.float64)})
    h = torch.tensor([[2.0, 0.0, 1.0]], dtype=torch.float64)
    # experts 0 and 1 give nothing; 1 is chosen by its correction, beside 0: the identity (2) is not
    assert float(P.experts_ff(W, "", {"router": {"experts": 2, "identity": 1, "top": 2}}, h).abs().max()) == 0.0
    W["correction"] = torch.tensor([0.0, -0.9, 0.0], dtype=torch.float64)
    share = math.exp(1) / (math.exp(2) + math.exp(1))
    assert torch.allclose(P.experts_ff(W, "", {"router": {"experts": 2, "identity": 1, "top": 2}}, h), share * h, atol=1e-12)
