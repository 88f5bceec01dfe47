"""Bafavik configurations as data, the sizes that only tensors tell, refusals, the states of runs, and the plain
implementation's pieces pinned against library routines."""
import copy

import pytest
import torch

from axon_amd.config import BafavikConfig, ConfigError, config_from_dict
from axon_amd.engine.loading import read_model_config
from axon_amd.models import build_model_description
from axon_amd.weights import Checkpoint, CheckpointSource, WeightError, check_tensors, write_random_model
from bafavik_models import MODELS, draw_weights, make, write_model
from plain import bafavik_plain as P


@pytest.mark.parametrize("name", sorted(MODELS))
def test_a_checkpoint_fits_what_the_parts_declare(name, tmp_path):
    folder = make(str(tmp_path), name)
    ck = Checkpoint(folder)
    cfg = read_model_config(folder, ck)
    assert isinstance(cfg, BafavikConfig) and cfg.to_dict() == MODELS[name]["cfg"]
    model = build_model_description(cfg)
    check_tensors(model.tensors(), CheckpointSource(ck), cfg.ignores_tensor)
    # the ranks come from the tensors' shapes
    for tensor, rank in MODELS[name]["rank"].items():
        delta = model.blocks[int(tensor[1])].mixer.sides[1]
        assert (delta.decay_rank if tensor.endswith("a1") else delta.gate_rank) == rank
    assert [r.layer for r in model.order] == P.run_order(cfg.cfg)


def test_constants_of_the_configuration_reach_the_parts():
    spec = config_from_dict(MODELS["A"]["cfg"]).model_spec()
    att, pair, pair2 = (L.mixer.params for L in spec.layers)
    assert (att["maps"], att["bias"], att["gate"], att["diff"], att["mask"], att["position"]) == (
        2, True, "elements", 0.3, {"kind": "chunk", "size": 7}, None)
    left, right = pair["left"].params, pair["right"].params
    assert pair["combine"] == "scaled" and pair["scales"] == [0.8, 0.9]
    assert left["position"].params["pairing"] == "halves" and left["qk_norm"] == "plain" and left["out_bias"] and right["decay"] == [0.5, 0.97]
    left, right = pair2["left"].params, pair2["right"].params
    assert pair2["combine"] == "normed" and pair2["mult"] == 0.5 and pair2["eps"] == 1e-5
    assert left["position"].params["pairing"] == "neighbours" and left["conv"] == 3 and left["gate"] == "elements" and not left.get("bias")
    assert right["gate_act"] == "sigmoid" and right["decay"] and right["gate"] and right["conv"] == 2
    assert spec.embedding.kind == "pair_embedding" and spec.embedding.params["scale"] == 1.5
    assert spec.embedding.params["pairs"] == {"tensor": "bigram", "buckets": 13, "mul_prev": 5, "mul_cur": 3}
    norm = spec.layers[0].norm.params
    assert (norm["residual_mult"], norm["layer_scale"], norm["token_shift"], norm["offset"]) == (0.7, True, True, 1.0)
    assert spec.head.params["scale"] == 1.5 and spec.layers[1].feed_forward is None
    assert spec.layers[0].feed_forward.params["activation"] == "relu_squared"
    assert config_from_dict(MODELS["C"]["cfg"]).model_spec().embedding.kind == "token_embedding"


def test_every_run_has_caches_and_states_of_its_own():
    model = build_model_description(config_from_dict(MODELS["A"]["cfg"]))
    plan = model.cache_plan
    assert [r.layer for r in model.order] == [0, 1, 2, 1, 2] and len({r.cache for r in model.order}) == 5
    held = [i for b in plan.bindings for i in (b.state_index, *b.more_states, b.block_state) if i >= 0]
    held.append(model.embedding.state_index)
    assert sorted(held) == list(range(len(plan.state_elems)))          # every arena belongs to one run, or the embedding
    # the attention of layer 2 keeps projections, its right side a matrix: two arenas; layer 1 only its right side's; layer 0 none
    assert [len([i for i in (b.state_index, *b.more_states) if i >= 0]) for b in plan.bindings] == [0, 1, 2, 1, 2]
    assert all(b.block_state >= 0 for b in plan.bindings) and plan.state_elems[model.embedding.state_index] == (2, "int32")
    assert plan.state_elems[plan.bindings[0].block_state] == (2 * 42, "float32")
    pair = plan.bindings[2]
    assert pair.with_states(1, 1).state_index == pair.more_states[0] and pair.with_states(0, 1).more_states == ()
    assert pair.with_states(0, 0).state_index == -1 and pair.with_states(1, 1).index == pair.index
    # one tap keeps nothing
    assert build_model_description(config_from_dict(MODELS["C"]["cfg"])).blocks[0].mixer.sides[0].state_specs() == []


def test_random_weights_round_trip(tmp_path):
    cfg = config_from_dict(MODELS["B"]["cfg"])
    folder = write_random_model(cfg, str(tmp_path / "m"), seed=3)
    back = read_model_config(folder)
    check_tensors(build_model_description(back).tensors(), CheckpointSource(Checkpoint(folder)))
    assert build_model_description(back).blocks[0].mixer.sides[1].decay_rank == 16


@pytest.mark.parametrize("edit,fragment", [
    (lambda c: c["layers"][0].update(type="delta"), "is not a mixer of this design"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "is not a feed-forward of this design"),
    (lambda c: c["layers"][0]["mixer"].update(heads=3), "not a multiple of"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "at least 1"),
    (lambda c: c["layers"][0]["mixer"].pop("diff"), "missing diff"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(decay=[0.5]), "has 1 numbers for 2 heads"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(decay="slow"), "not a list of numbers"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(dim=300), "takes 1 to 256"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=3), "must be even"),
    (lambda c: c["layers"][1]["mixer"].pop("left"), "is not an object"),
    (lambda c: c["layers"][2]["mixer"]["right"].update(kv_heads=2), "not a multiple of"),
    (lambda c: c["layers"][2]["mixer"]["left"].update(conv=0), "at least 1"),
    (lambda c: c["embedding"]["bigram"].update(buckets=0), "at least 1"),
    (lambda c: c["embedding"]["bigram"].update(mul_prev=1 << 33), "not a whole number"),
    (lambda c: c["loop"].update(stop=4), "of 3"),
    (lambda c: c.update(layers=[]), "not a list of layers"),
    (lambda c: c.pop("norm"), "is not an object"),
])
def test_refusals(edit, fragment):
    cfg = copy.deepcopy(MODELS["A"]["cfg"])
    edit(cfg)
    with pytest.raises(ConfigError, match=fragment):
        build_model_description(config_from_dict(cfg))


def test_missing_tensors_are_reported_together(tmp_path):
    m = MODELS["E"]
    W = draw_weights(m["cfg"], 1, m["rank"])
    gone = {"l1.mix.right.a1", "l1.mix.left.k.conv", "l0.shift", "l1.ls2", "bigram"}
    folder = write_model(str(tmp_path), m["cfg"], {k: v for k, v in W.items() if k not in gone})
    cfg = read_model_config(folder)
    with pytest.raises(WeightError) as e:
        check_tensors(build_model_description(cfg).tensors(), CheckpointSource(Checkpoint(folder)))
    assert gone <= set(e.value.missing)


# --------------------------------------------------------------------------- pins of the plain implementation
def test_the_plain_attention_is_a_library_attention():
    g = torch.Generator().manual_seed(1)
    q, k, v = (torch.randn(9, n, 6, generator=g, dtype=torch.float64) for n in (4, 2, 2))
    rep = lambda x: x.repeat_interleave(2, dim=1).transpose(0, 1)
    library = lambda **kw: torch.nn.functional.scaled_dot_product_attention(q.transpose(0, 1), rep(k), rep(v), scale=0.3, **kw).transpose(0, 1)
    assert torch.allclose(P.heads_attention(q, k, v, 0.3, None), library(is_causal=True), atol=1e-12)
    # chunks of four: three attentions of their own
    blocks = torch.block_diag(*[torch.ones(n, n).tril() for n in (4, 4, 1)]).bool()
    assert torch.allclose(P.heads_attention(q, k, v, 0.3, {"size": 4}), library(attn_mask=blocks), atol=1e-12)


def test_the_plain_recurrences_reduce_to_sums():
    g = torch.Generator().manual_seed(2)
    q, k, v = (torch.randn(7, 2, 4, generator=g, dtype=torch.float64) for _ in range(3))
    decay = torch.tensor([0.5, 0.9], dtype=torch.float64)
    got = P.lightning_recurrence(q, k, v, decay)
    for t in range(7):
        want = sum(decay[:, None] ** (t - s) * (q[t] * k[s]).sum(-1, keepdim=True) * v[s] for s in range(t + 1))
        assert torch.allclose(got[t], want, atol=1e-12)
    # the delta rule on orthonormal keys with beta 1 stores what it is given, row by row decayed, and a key met again
    # replaces its value
    eye = torch.eye(4, dtype=torch.float64)
    keys = eye[[0, 1, 2, 0]][:, None, :]
    vals = torch.randn(4, 1, 3, generator=g, dtype=torch.float64)
    one = torch.ones(4, 1, dtype=torch.float64)
    w = torch.tensor([0.5, 0.25, 1.0, 0.1], dtype=torch.float64).expand(4, 1, 4)
    assert torch.allclose(P.delta_recurrence(keys, keys, vals, w, one), vals, atol=1e-12)
    reads = P.delta_recurrence(eye[[3, 0, 0, 1]][:, None, :], keys, vals, w, one)
    assert torch.allclose(reads[3], vals[1] * 0.25 ** 2, atol=1e-12) and torch.allclose(reads[2], vals[0] * 0.5 ** 2, atol=1e-12)
    assert float(reads[0].abs().max()) == 0.0


def test_the_plain_rotation_is_a_complex_product():
    g = torch.Generator().manual_seed(3)
    v = torch.randn(5, 2, 10, generator=g, dtype=torch.float64)
    turn = torch.exp(1j * torch.arange(5)[:, None].double() * 50.0 ** (-2.0 * torch.arange(3).double() / 6))[:, None, :]
    z = torch.complex(v[..., :3], v[..., 3:6]) * turn
    assert torch.allclose(P.rotated(v, {"dims": 6, "base": 50.0}, False), torch.cat([z.real, z.imag, v[..., 6:]], -1), atol=1e-12)
    z = torch.complex(v[..., 0:6:2], v[..., 1:6:2]) * turn
    want = torch.cat([torch.view_as_real(z).flatten(-2), v[..., 6:]], -1)
    assert torch.allclose(P.rotated(v, {"dims": 6, "base": 50.0}, True), want, atol=1e-12)


def test_the_plain_small_pieces_are_library_ones():
    g = torch.Generator().manual_seed(4)
    x = torch.randn(9, 8, generator=g, dtype=torch.float64)
    assert torch.allclose(P.unit(x, 0.1), torch.nn.functional.rms_norm(x, (8,), eps=0.1), atol=1e-12)
    assert torch.allclose(P.softplus(x), torch.nn.functional.softplus(x), atol=1e-9)
    assert torch.allclose(P.silu(x), torch.nn.functional.silu(x), atol=1e-12)
    w = torch.randn(8, 3, generator=g, dtype=torch.float64)
    padded = torch.nn.functional.pad(x.T[None], (2, 0))
    assert torch.allclose(P.causal_conv(x, w), torch.nn.functional.conv1d(padded, w[:, None], groups=8)[0].T, atol=1e-12)
    share = torch.rand(8, generator=g, dtype=torch.float64)
    assert torch.allclose(P.shifted(x, share)[1:], torch.lerp(x[1:], x[:-1], share), atol=1e-12)
    assert torch.allclose(P.shifted(x, share)[0], x[0] * (1 - share), atol=1e-12)
    assert P.bigram_rows([4, 9, 9], {"buckets": 10, "mul_prev": 3, "mul_cur": 2}) == [10, (12 + 18) % 10, (27 + 18) % 10]
