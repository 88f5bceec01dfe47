"""The Bafavik decoder through the engine against the plain implementation (tests/plain/bafavik_plain.py): whole prompts,
decoding token by token from the first token on, portions down to two tokens, unequal requests side by side with pages, slots
and states that come round again, long stretches and long decoding, generation through the engine's own entry point (with
pages running out as well), the command line, the trace replay program, and every mechanism alone with weights or inputs made
so that a fault shows (a chunk one position off, a far key lost, a state, a convolution or a shift not carried across a cut, a
wrong row of the token pairs: each differs from the plain implementation by far more than the tolerance)."""
import math
import os
import subprocess
import sys

import pytest
import torch

import axon_amd
from axon_amd.config import config_from_dict
from axon_amd.config.base import PartSpec
from axon_amd.engine import Runtime, StepEntry
from axon_amd.kernels import KernelError
from axon_amd.parts import CacheBinding, build_part
from axon_amd.weights import WeightStore
from bafavik_models import MODELS, config, diff_att, draw_weights, heads, layer, make, parallel, parallel_2, rot
from gpu_helpers import DTYPES, DictSource, PartHarness
from helpers import ROOT, TraceBuilder, engine_for, run_trace, tolerance
from plain import bafavik_plain as P

pytestmark = pytest.mark.gpu


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            made[name] = make(str(tmp_path_factory.mktemp("bafavik_" + name)), name)
        return made[name]
    return get


@pytest.fixture(scope="module")
def plain_logits(folders):
    kept, models = {}, {}

    def get(name, seq):
        if name not in models:
            models[name] = P.load_plain(folders(name))
        key = (name, tuple(seq))
        if key not in kept:
            kept[key] = P.forward_logits(*models[name], seq).float()
        return kept[key]
    return get


def sequences(name, lengths, seed=0):
    g = torch.Generator().manual_seed(seed)
    return [torch.randint(0, MODELS[name]["cfg"]["vocab"], (n,), generator=g).tolist() for n in lengths]


def assert_close(got, ref, dtype, what):
    """Rows of logits against the plain implementation's.  32-bit: every row within rounding.  16 bits: a head's output is
    divided by its root mean square, and a row whose output happens to be small passes its rounding on many times enlarged;
    so one row in fifty may reach twice the limit of the others."""
    err = (got - ref).abs().max(dim=-1).values
    limit = tolerance(dtype, ref) * (2.0 if dtype == "float32" else 3.0)
    if dtype == "float32":
        assert float(err.max()) <= limit, f"{what}: {float(err.max())} > {limit} at row {int(err.argmax())}"
        return
    over = int((err > limit).sum())
    assert over <= max(1, len(err) // 50) and float(err.max()) <= 2 * limit, \
        f"{what}: {over} of {len(err)} rows over {limit}, the worst {float(err.max())} at row {int(err.argmax())}"


def run_schedule(eng, seqs, schedule):
    """schedule: steps of [(request, tokens)]; every position's logits are asked for.  A request ends with its last token.
    Returns {request: [len, vocab]}."""
    at = {r: 0 for r in seqs}
    got = {r: [] for r in seqs}
    for step in schedule:
        entries, ends = [], []
        for rid, n in step:
            toks = seqs[rid][at[rid]:at[rid] + n]
            entries.append(StepEntry(rid, toks, list(range(len(toks)))))
            at[rid] += len(toks)
            if at[rid] == len(seqs[rid]):
                ends.append(rid)
        out = eng.step(entries, ends).cpu()
        row = 0
        for e in entries:
            got[e.id].append(out[row:row + len(e.tokens)].clone())
            row += len(e.tokens)
    assert all(at[r] == len(seqs[r]) for r in seqs)
    return {r: torch.cat(v) for r, v in got.items()}


def pages_for(name, tokens):
    return -(-tokens // MODELS[name]["page"]) + 2


# --------------------------------------------------------------------------- whole models
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MODELS))
def test_whole_prompts_and_decoding_token_by_token(folders, plain_logits, name, dtype):
    n = 200 if name == "B" else 90
    (seq,) = sequences(name, [n], seed=1)
    ref = plain_logits(name, seq)
    eng = engine_for(folders(name), dtype, MODELS[name]["page"], pages_for(name, n), max_seqs=2, max_seq_len=256)
    whole = run_schedule(eng, {"a": seq}, [[("a", n)]])["a"]
    assert_close(whole, ref, dtype, "whole prompt")
    # from the first token on, one token a step: the first tokens of a sequence (states, shifts, convolutions and token
    # pairs that start from nothing), every page's edge, every chunk's edge
    single = run_schedule(eng, {"b": seq}, [[("b", 1)] for _ in range(n)])["b"]
    assert_close(single, ref, dtype, "token by token")
    # most of it at once, the rest decoded
    got = run_schedule(eng, {"c": seq}, [[("c", n - 45)]] + [[("c", 1)] for _ in range(45)])["c"]
    assert_close(got, ref, dtype, "prompt then decoding")
    if dtype == "float32":
        assert float((single - whole).abs().max()) <= 2 * tolerance(dtype, ref)
    eng.cache.check()


def test_what_the_whole_models_would_catch(folders):
    """Mistakes of a layer's arrangement, planted in the plain implementation: each moves the logits by far more than the
    tests above allow."""
    name = "A"
    cfg, W = P.load_plain(folders(name))
    (seq,) = sequences(name, [40], seed=1)
    ref = P.forward_logits(cfg, W, seq).float()
    loud = 20 * tolerance("float32", ref)
    logits = lambda c=cfg, w=W: P.forward_logits(c, w, seq).float()
    moved = lambda got: float((got - ref).abs().max()) > loud
    for key in ("l0.shift", "l1.shift", "l0.ls1", "l0.ls2", "l1.ls1", "l2.mix.left.out", "l1.mix.left.o.b", "final.norm", "l2.norm2"):
        assert moved(logits(w=dict(W, **{key: torch.zeros_like(W[key]) + (1.0 if ".ls" in key else 0.0)}))), key
    for edit in (dict(residual_mult=0.5), dict(logit_scale=1.0), dict(loop={"start": 1, "stop": 3, "times": 1}),
                 dict(embedding=dict(cfg["embedding"], scale=1.0)), dict(embedding={"scale": 1.5}),
                 dict(embedding=dict(cfg["embedding"], bigram={"buckets": 13, "mul_prev": 3, "mul_cur": 5}))):
        assert moved(logits(c=dict(cfg, **edit))), edit
    # the first token: its own row of the token pairs, and a shift towards zeros
    rows, shifted = P.bigram_rows, P.shifted
    try:
        P.bigram_rows = lambda t, b: [(t[0] * b["mul_cur"]) % b["buckets"]] + rows(t, b)[1:]
        assert moved(logits())
        P.bigram_rows = rows
        P.shifted = lambda h, share: torch.cat([h[:1], shifted(h, share)[1:]])
        assert moved(logits())
    finally:
        P.bigram_rows, P.shifted = rows, shifted


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MODELS))
def test_portions_of_many_sizes_down_to_two_tokens(folders, plain_logits, name, dtype):
    n = 220 if name == "B" else 90
    (seq,) = sequences(name, [n], seed=2)
    eng = engine_for(folders(name), dtype, MODELS[name]["page"], pages_for(name, n), max_seqs=2, max_seq_len=256)
    for cuts in ([2, 2, 3, 1, 2, 7, 1, 1, 5, 64, 2], [63, 2, 1, 64, 9], [8, 8, 1, 16, 2]):
        sched, rest, i = [], n, 0
        while rest:
            take = min(cuts[i % len(cuts)], rest)
            sched.append([("a", take)])
            rest -= take
            i += 1
        assert_close(run_schedule(eng, {"a": seq}, sched)["a"], plain_logits(name, seq), dtype, f"portions {cuts}")
    eng.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MODELS))
def test_unequal_requests_side_by_side_with_pages_and_slots_used_again(folders, plain_logits, name, dtype):
    lengths = [57, 5, 120, 33, 1, 76]
    seqs = dict(enumerate(sequences(name, lengths, seed=3)))
    page = MODELS[name]["page"]
    # three slots and a pool for the three longest live at once: later requests get the pages, the slots and
    # the state rows of finished ones
    eng = engine_for(folders(name), dtype, page, 3 * (-(-120 // page)) + 1, max_seqs=3, max_seq_len=128, shuffle_pages_seed=5)
    cuts = {0: [9, 1, 1, 2, 30, 1], 1: [2, 1, 1, 1], 2: [1, 40, 1, 1, 3, 64, 1], 3: [33], 4: [1], 5: [2, 1, 50, 1, 1, 1]}
    at = {r: 0 for r in seqs}
    waiting, live, sched, turn = [0, 1, 2, 3, 4, 5], [], [], 0
    while waiting or live:
        while waiting and len(live) < 3:
            live.append(waiting.pop(0))
        step = []
        for r in list(live):
            if (turn + r) % 4 == 3 and len(live) > 1:
                continue                                  # left out of this step, goes on later
            n = min(cuts[r][(turn // 2) % len(cuts[r])], lengths[r] - at[r])
            step.append((r, n))
            at[r] += n
            if at[r] == lengths[r]:
                live.remove(r)
        if step:
            sched.append(step)
        turn += 1
    got = run_schedule(eng, seqs, sched)
    for r in seqs:
        assert_close(got[r], plain_logits(name, seqs[r]), dtype, f"request {r} in the mixed schedule")
    eng.cache.check()
    assert not eng.live
    for g in range(len(eng.cache.groups)):
        assert eng.cache.free_pages(g) == eng.cache.groups[g].n_pages
    if dtype == "float32":
        # each request alone gives the same rows as side by side, to rounding
        alone = run_schedule(eng, {2: seqs[2]}, [[(2, lengths[2])]])
        assert float((alone[2] - got[2]).abs().max()) <= 2 * tolerance(dtype, plain_logits(name, seqs[2]))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B", "C", "E"])
def test_long_stretches_run_the_recurrences_in_chunks(folders, plain_logits, name, dtype):
    """Hundreds of tokens of a request in one step: where the sizes allow, the recurrences run in chunks on the matrix cores;
    the states they leave are what later portions and decoded tokens go on from.  Beside a short request in the same step.  A
    stretch of an even number of tokens ends in the copy of the states that it started from, one of an odd number in the other."""
    n = 721
    long, short = sequences(name, [n, 9], seed=5)
    page = MODELS[name]["page"]
    eng = engine_for(folders(name), dtype, page, -(-n // page) + 4, max_seqs=2, max_seq_len=768, max_batch_tokens=544)
    chunked = {"delta_scan": [], "lightning_scan": []}
    for entry, seen in chunked.items():
        def logged(*a, _inner=getattr(eng.rt.k, entry), _seen=seen, chunks=None, **kw):
            _seen.append(chunks is not None)
            return _inner(*a, chunks=chunks, **kw)
        setattr(eng.rt.k, entry, logged)
    try:
        got = run_schedule(eng, {"a": long, "b": short}, [[("a", 530), ("b", 4)], [("a", 1), ("b", 5)], [("a", 2)], [("a", 187)], [("a", 1)]])
    finally:
        for entry in chunked:
            delattr(eng.rt.k, entry)
    for entry, seen in chunked.items():
        assert not all(seen) and any(seen) == (name in ("B", "E")), (entry, seen)
    assert_close(got["a"], plain_logits(name, long), dtype, "the long request")
    assert_close(got["b"], plain_logits(name, short), dtype, "the short request beside it")
    eng.cache.check()


@pytest.mark.parametrize("name", ["A", "C", "D"])
def test_long_decoding_across_many_pages(folders, plain_logits, name):
    n = 250
    (seq,) = sequences(name, [n], seed=4)
    eng = engine_for(folders(name), "float32", MODELS[name]["page"], pages_for(name, n), max_seqs=1, max_seq_len=256)
    got = run_schedule(eng, {"a": seq}, [[("a", 3)]] + [[("a", 1)] for _ in range(n - 3)])
    assert_close(got["a"], plain_logits(name, seq), "float32", "long decoding")


@pytest.mark.parametrize("name", sorted(MODELS))
def test_greedy_generation_through_the_entry_point(folders, name):
    cfg, W = P.load_plain(folders(name))
    prompts = sequences(name, [11, 3, 30], seed=6)
    want = [P.greedy_generate(cfg, W, p, 10) for p in prompts]
    page = MODELS[name]["page"]
    pages = 3 * (-(-128 // page))
    llm = axon_amd.load(folders(name), dtype="float32", page_size=page, num_pages=pages, max_seqs=3, max_seq_len=128)
    assert llm.generate(prompts, max_new_tokens=10) == want                       # decoding steps replay graphs
    assert llm.engine.graphs_ok and all(c for c, _, _ in llm.engine._segments)
    assert llm.generate(prompts[:1], max_new_tokens=10) == want[:1]               # alone, in a slot used before
    eager = axon_amd.load(folders(name), dtype="float32", page_size=page, num_pages=pages, max_seqs=3, max_seq_len=128,
                          use_graphs=False)
    assert eager.generate(prompts, max_new_tokens=10) == want
    # 16 bits: the tokens that come out of the scheduler's steps and the graphs are the best of the engine's own
    # logits of prompt and tokens in one step (what those logits are worth is the matter of the tests above)
    half = axon_amd.load(folders(name), dtype="bfloat16", page_size=page, num_pages=pages, max_seqs=3, max_seq_len=128)
    for p, o in zip(prompts, half.generate(prompts, max_new_tokens=10)):
        logits = half.logits(p + o, all_positions=True).float().cpu()
        for i, tok in enumerate(o):
            row = logits[len(p) - 1 + i]
            assert float(row.max() - row[tok]) <= tolerance("bfloat16", logits)


@pytest.mark.parametrize("dtype", DTYPES)
def test_replayed_decoding_steps_give_the_eager_bits(folders, dtype):
    """The same requests decoded for many steps once from graphs and once launch by launch: equal bits, step for step."""
    name = "B"
    seqs = dict(enumerate(sequences(name, [70, 41], seed=14)))
    rows = {}
    for graphs in (False, True):
        eng = engine_for(folders(name), dtype, 64, 8, max_seqs=2, max_seq_len=128, use_graphs=graphs)
        rows[graphs] = run_schedule(eng, seqs, [[(0, 40), (1, 11)]] + [[(0, 1), (1, 1)] for _ in range(30)])
    for r in seqs:
        assert torch.equal(rows[False][r], rows[True][r])


@pytest.mark.parametrize("name", ["A", "D"])
def test_generation_goes_on_where_pages_run_out(folders, name):
    """A pool that three requests outgrow while they generate: the youngest gives up its pages and its states, and is fed
    again later; the tokens are those of a roomy pool."""
    page = MODELS[name]["page"]
    prompts = sequences(name, [2 * page, 2 * page - 3, page + 1], seed=8)
    load = lambda pages: axon_amd.load(folders(name), dtype="float32", page_size=page, num_pages=pages, max_seqs=3, max_seq_len=128)
    want = load(64).generate(prompts, max_new_tokens=40)
    tight = load(-(-(2 * page + 40) // page) + 3)
    assert tight.generate(prompts, max_new_tokens=40) == want
    assert tight.last_stats.preemptions > 0
    tight.engine.cache.check()


def test_the_command_line_generates_with_the_design(folders):
    name = "E"
    cfg, W = P.load_plain(folders(name))
    p, q = sequences(name, [9, 14], seed=9)
    axon = [sys.executable, os.path.join(ROOT, "bin", "axon")]
    ids = lambda seq: " ".join(map(str, seq))
    r = subprocess.run(axon + ["gen", folders(name), ids(p), ids(q), "-n", "8", "--dtype", "float32", "--page-size", "64"],
                       capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr
    assert [[int(t) for t in line.split()] for line in r.stdout.splitlines()] == [
        P.greedy_generate(cfg, W, p, 8), P.greedy_generate(cfg, W, q, 8)]


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_trace_replay_program_runs_the_design(folders, plain_logits, tmp_path, dtype):
    name = "B"
    seqs = sequences(name, [40, 17, 64], seed=7)
    refs = [plain_logits(name, s) for s in seqs]
    tb = TraceBuilder()
    tb.step([("a", seqs[0][:30], [0, 29]), ("b", seqs[1][:2], [1])])
    tb.step([("a", seqs[0][30:31], [0]), ("b", seqs[1][2:], [0, 14]), ("c", seqs[2][:7], [])], end=["b"])
    tb.step([("a", seqs[0][31:], [8]), ("c", seqs[2][7:], [0, 56])], end=["a", "c"])
    rows = tb.collect(run_trace(folders(name), dtype, tb.steps, str(tmp_path), max_tokens=192))
    for (rid, pos), row in rows.items():
        ref = refs["abc".index(rid)]
        assert float((torch.from_numpy(row) - ref[pos]).abs().max()) <= 3 * tolerance(dtype, ref)


# --------------------------------------------------------------------------- the mechanisms alone
def rows_in(T, width, seed, dtype, scale=1.0):
    """Random rows; for the 16-bit run, rows that 16 bits hold exactly (the plain run starts from the same numbers)."""
    g = torch.Generator().manual_seed(seed)
    h = torch.randn(T, width, generator=g) * scale
    return h.to(torch.bfloat16).float() if dtype == "bfloat16" else h


def part_tol(dtype, ref):
    return (3e-5 if dtype == "float32" else 3e-2) * max(1.0, float(ref.abs().max()))


def mixer_of(cfg, side=None, ranks=None):
    """The mixer of layer 0, or one side of it."""
    c = config_from_dict(cfg)
    if ranks:
        c = c.with_sizes({name: (rank, cfg["width"]) for name, rank in ranks.items()})
    spec = c.layers[0]["mixer"]
    if side is not None:
        spec = spec.params[side]
    return build_part("mixer", spec, "l0.")


def harness_for(part, dtype, page, T):
    return PartHarness(dtype, part.cache_spec(), page_size=page, n_pages=-(-T // page) + 3, max_seq_len=1024,
                       state_elems=[(s.elems, s.dtype) for s in part.state_specs()])


def run_mixer(part, W, harness, h, cuts, width, **kw):
    """The mixer's 32-bit output for rows h, fed in portions of the given sizes."""
    part.load(WeightStore(DictSource(W), harness.rt.device, harness.rt.dtype), harness.rt)
    n_states = len(part.state_specs())
    binding = CacheBinding(group=0, index=0, writes=True, state_index=0, more_states=tuple(range(1, n_states)))
    outs, at = [], 0
    for n in cuts:
        ctx = harness.ctx([0] * n)
        x = h[at:at + n].to(harness.rt.dtype).cuda()
        out = torch.full((n, width), 0.0 if kw.get("accumulate") else float("nan"), dtype=torch.float32, device="cuda")
        if kw.get("accumulate"):
            part.forward(ctx, binding, x, out)
        else:
            part.forward(ctx, binding, x, out, accumulate=False)
        outs.append(out.cpu())
        at += n
    assert at == h.shape[0]
    return torch.cat(outs)


CUTS = lambda T, page: [[T], [page - 1] + [1] * 8 + [T - page - 7], [2, 1, 1, 3] + [1] * 30 + [64, 2, T - 103], [1] * T]


def check_mixer(cfg, W, plain, dtype, T, cut_sets, side=None, ranks=None, page=16, h=None, rows=slice(None), **kw):
    h = rows_in(T, cfg["width"], 13, dtype) if h is None else h
    ref = plain(W, h).float()
    for cuts in cut_sets:
        part = mixer_of(cfg, side, ranks)
        got = run_mixer(part, W, harness_for(part, dtype, page, T), h, cuts, cfg["width"], **kw)
        err = (got - ref)[rows].abs().max(dim=-1).values
        # 16 bits: a row whose head happens to come out small passes its rounding on enlarged
        assert float(err.max()) <= part_tol(dtype, ref) * (1 if dtype == "float32" else 3), (cuts[:8], float(err.max()), int(err.argmax()))
        assert float(err.median()) <= part_tol(dtype, ref), (cuts[:8], float(err.median()))
    return h, ref


def doubles(W):
    return {k: v.double() for k, v in W.items()}


def weights_of(cfg, seed, ranks=None, scope="l0.mix."):
    return {k: v for k, v in draw_weights(cfg, seed, ranks).items() if k.startswith(scope)}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("h_n,dim,vdim", [(3, 5, 7), (2, 64, 32), (1, 132, 24), (4, 16, 16), (2, 256, 48), (8, 128, 128), (2, 48, 80),
                                          (1, 1, 1), (3, 200, 9), (2, 112, 272), (1, 8, 515)])
def test_linear_attention_alone_in_portions(h_n, dim, vdim, dtype):
    """The walk (and, where the sizes allow, the chunks) with its state carried across cuts of every kind: whole, a token at a
    time from the first token on, portions down to one token.  Decays from none left to none lost."""
    width, T = 48, 140
    decay = [0.97, 1.0, 0.3, 0.9995, 0.75, 1e-30, 0.6, 0.99][:h_n]
    cfg = config(width, 16, [layer(parallel(heads(1, 1, 8, 8), decay, dim, vdim), None)], eps=1e-3)
    W = weights_of(cfg, 41, scope="l0.mix.right.")
    c = cfg["layers"][0]["mixer"]["right"]
    plain = lambda W, h, c=c: P.lightning_mixer(doubles(W), "l0.mix.right.", c, h.double(), 1e-3)
    h, ref = check_mixer(cfg, W, plain, dtype, T, CUTS(T, 16), "right")
    # what the test would catch: a state that starts anew at a cut, a read before the write, decays, norm per head, the gate
    loud = 20 * part_tol("float32", ref)
    moved = lambda got: float((got.float() - ref).abs().max()) > loud
    assert float((torch.cat([plain(W, h[:100]), plain(W, h[100:])]).float() - ref)[100:].abs().max()) > loud
    assert moved(plain(W, h, dict(c, decay=[0.9 * d for d in decay])))
    rule = P.lightning_recurrence
    try:
        P.lightning_recurrence = lambda q, k, v, d: rule(q, k, v, d) - (q * k).sum(-1, keepdim=True) * v
        assert moved(plain(W, h))
    finally:
        P.lightning_recurrence = rule
    unit = P.unit
    if h_n > 1:
        try:
            P.unit = lambda x, eps: unit(x.view(len(x), h_n, vdim), eps).reshape(len(x), -1)
            assert moved(plain(W, h))
        finally:
            P.unit = unit


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("h_n,kv,dim,vdim,conv,ranks", [
    (3, 1, 5, 7, 3, (3, 5)), (4, 2, 64, 32, 4, (16, 64)), (2, 2, 132, 24, 1, (1, 2)), (1, 1, 16, 40, 5, (70, 130)), (6, 3, 200, 16, 2, (7, 3)),
    (4, 4, 128, 128, 4, (64, 16)), (2, 1, 32, 72, 4, (6, 6)), (4, 4, 6, 9, 2, (9, 1)), (3, 3, 96, 80, 3, (20, 33)), (6, 2, 32, 16, 2, (8, 8))])
def test_the_delta_rule_with_a_decay_a_channel_alone_in_portions(h_n, kv, dim, vdim, conv, ranks, dtype):
    """The walk (and the chunks) with its state and the convolutions' kept inputs carried across cuts of every kind: whole, a
    token at a time from the first token on, portions that end inside the convolutions' reach."""
    width, T = 48, 140
    cfg = config(width, 16, [layer(parallel_2(heads(1, 1, 8, 8), 2, h_n, kv, dim, vdim, conv), None)], eps=1e-3)
    names = {"l0.mix.right.a1": ranks[0], "l0.mix.right.g1": ranks[1]}
    W = weights_of(cfg, 43, names, "l0.mix.right.")
    c = cfg["layers"][0]["mixer"]["right"]
    plain = lambda W, h: P.delta_mixer(doubles(W), "l0.mix.right.", c, h.double(), 1e-3)
    h, ref = check_mixer(cfg, W, plain, dtype, T, CUTS(T, 16), "right", names)
    loud = 20 * part_tol("float32", ref)
    moved = lambda got: float((got.float() - ref).abs().max()) > loud
    assert float((torch.cat([plain(W, h[:100]), plain(W, h[100:])]).float() - ref)[104:].abs().max()) > loud
    # no decay, one decay a head (the channels' mean), the decay behind the correction, keys that are not of length 1
    rule, length = P.delta_recurrence, P.unit_length
    try:
        P.delta_recurrence = lambda q, k, v, g, beta: rule(q, k, v, torch.ones_like(g), beta)
        assert moved(plain(W, h))
        P.delta_recurrence = lambda q, k, v, g, beta: rule(q, k, v, g.mean(-1, keepdim=True).expand_as(g), beta)
        assert moved(plain(W, h))
        P.delta_recurrence = lambda q, k, v, g, beta: rule(q, k, v, torch.cat([torch.ones_like(g[:1]), g[:-1]]), beta)
        assert moved(plain(W, h))
        P.delta_recurrence = rule
        P.unit_length = lambda x: x
        assert moved(plain(W, h))
    finally:
        P.delta_recurrence, P.unit_length = rule, length
    for name in ("dt_bias", "g2", "a2"):
        assert moved(plain(dict(W, **{"l0.mix.right." + name: torch.zeros_like(W["l0.mix.right." + name])}), h)), name


@pytest.mark.parametrize("T", [64, 65, 100, 128, 200])
def test_chunks_with_decays_that_vanish(T):
    """Decays of exactly 0, of 1e-30 and of 1 side by side in the chunks of the delta rule and of linear attention: products of
    decays underflow to nothing, and nothing is divided by them."""
    rt = Runtime("float32")
    h_n, kv, N, P_n, g = 2, 1, 64, 32, torch.Generator().manual_seed(T)
    q, k = (P.unit_length(torch.randn(T, kv, N, generator=g).double()) for _ in range(2))
    v, beta = torch.randn(T, h_n, P_n, generator=g).double(), torch.rand(T, h_n, generator=g).double()
    w = torch.rand(T, h_n, N, generator=g).double()
    w[:, :, 0::4], w[:, 0, 1::4], w[5::7, 1, 2::4] = 1.0, 1e-30, 0.0
    want = P.delta_recurrence(q.repeat(1, h_n, 1), k.repeat(1, h_n, 1), v, w, beta).reshape(T, -1)
    u = torch.cat([q.reshape(T, -1), k.reshape(T, -1), v.reshape(T, -1)], 1).float().cuda()
    terms = torch.stack([torch.ones(T, h_n), beta.float()], -1).contiguous().cuda()
    copy = h_n * N * P_n
    i32 = lambda rows: torch.tensor(rows, dtype=torch.int32).cuda()
    chunks = i32([[at, min(64, T - at)] for at in range(0, T, 64)])
    arguments = (i32(list(range(T))), i32([0] * T))
    y = torch.full((T, h_n * P_n), float("nan"), device="cuda")
    state = torch.zeros(1, 2 * copy, device="cuda")
    rt.k.delta_scan(u, terms, state, copy, copy, i32([]).view(0, 3), *arguments, u, y, h_n, kv, N, P_n, 1,
                    chunks=(chunks, i32([[0, 0, T, 0, len(chunks)]])), decay=w.float().reshape(T, -1).contiguous().cuda())
    assert float((y.cpu().double() - want).abs().max()) <= 2e-5 * float(want.abs().max())
    walked, y2 = torch.zeros(1, 2 * copy, device="cuda"), torch.empty_like(y)
    rt.k.delta_scan(u, terms, walked, copy, copy, i32([[0, 0, T]]), *arguments, u, y2, h_n, kv, N, P_n, 1,
                    decay=w.float().reshape(T, -1).contiguous().cuda())
    assert float((y2.cpu().double() - want).abs().max()) <= 2e-5 * float(want.abs().max())
    assert float((state - walked).abs().max()) <= 2e-5 * float(walked.abs().max())
    # linear attention: a head whose decay is 0, one at 1
    rows = torch.randn(T, 2 * h_n * N + h_n * P_n, generator=g)
    decay = torch.tensor([0.0, 1.0])
    split = rows.double().split([h_n * N, h_n * N, h_n * P_n], 1)
    want = P.lightning_recurrence(*(x.view(T, h_n, -1) for x in split), decay.double()).reshape(T, -1)
    state = torch.zeros(1, 2 * copy, device="cuda")
    rt.k.lightning_scan(rows.cuda(), 0, h_n * N, 2 * h_n * N, False, decay.cuda(), state, copy, i32([]).view(0, 3), *arguments, y, h_n, N, P_n,
                        chunks=(chunks, i32([[0, 0, T, 0, len(chunks)]])))
    assert float((y.cpu().double() - want).abs().max()) <= 2e-5 * float(want.abs().max())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["linear", "delta"])
def test_a_slow_state_remembers_an_input_hundreds_of_positions_back(kind, dtype):
    """Decays of 0.999 a step, a loud row at position 3 and rows that write nothing (or faintly) after it: 600 positions on, the
    output is still that row's doing, in a prompt and decoded one token at a time."""
    width, T, ranks = 32, 640, None
    if kind == "linear":
        cfg = config(width, 16, [layer(parallel(heads(1, 1, 8, 8), [0.999], 16, 16), None)], eps=1e-3)
        W = weights_of(cfg, 43, scope="l0.mix.right.")
        c = cfg["layers"][0]["mixer"]["right"]
        plain = lambda W, h: P.lightning_mixer(doubles(W), "l0.mix.right.", c, h.double(), 1e-3)
    else:
        ranks = {"l0.mix.right.a1": 4, "l0.mix.right.g1": 4}
        cfg = config(width, 16, [layer(parallel_2(heads(1, 1, 8, 8), 1, 1, 1, 64, 16, 2), None)], eps=1e-3)
        W = weights_of(cfg, 43, ranks, "l0.mix.right.")
        W["l0.mix.right.A_log"] = torch.tensor([math.log(0.001)])
        W["l0.mix.right.dt_bias"] = torch.full((64,), 0.5413)          # softplus gives 1: g = exp(-0.001)
        W["l0.mix.right.a2"] = torch.zeros_like(W["l0.mix.right.a2"])
        # the loud row writes, the faint ones read: a logit of beta that the loud row alone lifts
        W["l0.mix.right.b"] = torch.zeros_like(W["l0.mix.right.b"])
        W["l0.mix.right.b"][0, 0] = 4.0
        c = cfg["layers"][0]["mixer"]["right"]
        plain = lambda W, h: P.delta_mixer(doubles(W), "l0.mix.right.", c, h.double(), 1e-3)
    W = {k: v.to(torch.bfloat16).float() for k, v in W.items()}
    h = rows_in(T, width, 15, dtype, scale=0.05 if kind == "linear" else 1.0)
    h[3] = rows_in(1, width, 16, dtype, scale=3.0)[0]
    if kind == "delta":
        h[:, 0] = -3.0
        h[3, 0] = 3.0
    ref = plain(W, h).float()
    quiet = h.clone()
    quiet[3] = h[4]
    assert float((plain(W, quiet).float() - ref)[600:].abs().max()) > 0.2 * float(ref[600:].abs().max())
    check_mixer(cfg, W, plain, dtype, T, ([T], [600] + [1] * 40, [2, 3, 64, 129, 1, 1, 400, 38, 2]), "right", ranks, h=h, rows=slice(600, None))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("h_n,kv,dim,vdim,rt,page", [
    (3, 1, 10, 6, (4, 100.0), 8), (8, 2, 32, 32, (32, 100.0), 64), (4, 4, 64, 48, (32, 100.0), 64), (1, 1, 24, 40, None, 16),
    (6, 3, 48, 16, (48, 100.0), 128), (8, 2, 128, 256, (64, 100.0), 64), (4, 1, 256, 192, (128, 100.0), 64), (2, 2, 16, 272, (2, 9.0), 64)])
def test_attention_with_queries_and_keys_of_unit_size(h_n, kv, dim, vdim, rt, page, dtype):
    cfg = config(64, 16, [layer(parallel(heads(h_n, kv, dim, vdim, 1.7 / dim ** 0.5, **(rot(*rt) if rt else {})), [0.5], 4, 4), None)])
    W = weights_of(cfg, 31, scope="l0.mix.left.")
    c = cfg["layers"][0]["mixer"]["left"]
    plain = lambda W, h, c=c: P.turned_normed_attention(doubles(W), "l0.mix.left.", c, h.double(), 1e-5)
    T = 200
    h, ref = check_mixer(cfg, W, plain, dtype, T, CUTS(T, page)[:3], "left", page=page)
    loud = 20 * part_tol("float32", ref)
    moved = lambda got: float((got.float() - ref).abs().max()) > loud
    for name in ("q.b", "k.b", "v.b", "o.b"):
        assert moved(plain(dict(W, **{"l0.mix.left." + name: torch.zeros_like(W["l0.mix.left." + name])}), h)), name
    if rt is not None:
        assert moved(plain(W, h, dict(c, rot=None)))
        turn = P.rotated
        if rt[0] > 2:
            try:
                P.rotated = lambda v, r, neighbours: turn(v, r, not neighbours)
                assert moved(plain(W, h))
            finally:
                P.rotated = turn
    unit = P.unit
    try:
        P.unit = lambda x, eps: x
        assert moved(plain(W, h))
    finally:
        P.unit = unit


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("h_n,kv,dim,vdim,conv,rt,page", [
    (3, 1, 10, 6, 3, (4, 100.0), 8), (8, 2, 32, 32, 4, (32, 100.0), 64), (4, 4, 64, 48, 2, (32, 100.0), 64), (1, 1, 24, 40, 1, None, 16),
    (6, 3, 48, 16, 5, (48, 100.0), 128), (8, 2, 128, 128, 4, (64, 100.0), 64), (4, 1, 256, 192, 3, (128, 100.0), 64),
    (2, 1, 96, 256, 4, (96, 50.0), 64), (2, 2, 17, 9, 7, (16, 50.0), 32)])
def test_attention_behind_short_convolutions(h_n, kv, dim, vdim, conv, rt, page, dtype):
    """Portions that end inside the convolutions' reach, of even and odd sizes, and single tokens from the first one on."""
    cfg = config(64, 16, [layer(parallel_2(heads(h_n, kv, dim, vdim, **(rot(*rt) if rt else {})), conv, 1, 1, 4, 4, 1), None)])
    W = weights_of(cfg, 37, scope="l0.mix.left.")
    c = cfg["layers"][0]["mixer"]["left"]
    plain = lambda W, h, c=c: P.convolved_attention(doubles(W), "l0.mix.left.", c, h.double())
    T = 170
    h, ref = check_mixer(cfg, W, plain, dtype, T, CUTS(T, page)[:3] + [[2] * 30 + [1, 3] * 10 + [T - 100], [1] * T], "left", page=page)
    loud = 20 * part_tol("float32", ref)
    moved = lambda got: float((got.float() - ref).abs().max()) > loud
    assert moved(plain(dict(W, **{"l0.mix.left.g": torch.zeros_like(W["l0.mix.left.g"])}), h))
    if conv > 1:
        whole = P.causal_conv
        try:       # a convolution that starts anew at a cut
            P.causal_conv = lambda x, w: torch.cat([whole(x[:100], w), whole(x[100:], w)])
            assert moved(plain(W, h))
            P.causal_conv = lambda x, w: whole(x, w.flip(1))
            assert moved(plain(W, h))
        finally:
            P.causal_conv = whole
    if rt is not None and rt[0] > 2:
        turn = P.rotated
        try:
            P.rotated = lambda v, r, neighbours: turn(v, r, not neighbours)
            assert moved(plain(W, h))
        finally:
            P.rotated = turn


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("h_n,kv,dim,vdim,chunk,diff,page", [
    (3, 1, 10, 6, 7, 0.3, 8), (8, 2, 32, 32, 70, 0.1, 64), (4, 1, 56, 112, 80, 0.8, 64), (1, 1, 24, 40, 1, 0.5, 16), (6, 3, 40, 16, 128, 0.0, 128),
    (4, 4, 64, 128, 64, 0.2, 64), (2, 2, 128, 256, None, 0.4, 64), (8, 4, 16, 48, 33, 0.6, 64)])
def test_differential_attention_in_chunks(h_n, kv, dim, vdim, chunk, diff, page, dtype):
    cfg = config(64, 16, [layer(diff_att(h_n, kv, dim, vdim, chunk=chunk, diff=diff), None)], eps=1e-4)
    W = weights_of(cfg, 39)
    c = cfg["layers"][0]["mixer"]
    plain = lambda W, h, c=c: P.differential_attention(doubles(W), "l0.mix.", c, h.double(), 1e-4)
    T = 200
    h, ref = check_mixer(cfg, W, plain, dtype, T, CUTS(T, page)[:3], page=page)
    loud = 20 * part_tol("float32", ref)
    moved = lambda got: float((got.float() - ref).abs().max()) > loud
    if chunk is not None:
        assert moved(plain(W, h, dict(c, mask={"size": chunk + 1}))) and moved(plain(W, h, dict(c, mask=None)))
    assert moved(plain(W, h, dict(c, diff=diff + 0.1)))
    for name in ("q.b", "v.b", "lq1", "lk2", "g"):
        if chunk == 1 and name in ("q.b", "lq1", "lk2"):
            continue                                        # one key a row: the maps agree
        assert moved(plain(dict(W, **{"l0.mix." + name: torch.zeros_like(W["l0.mix." + name])}), h)), name


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["normed", "convolved"])
def test_a_key_hundreds_of_positions_back_decides_a_row(kind, dtype):
    """Weights set by hand: queries and keys read the same places of the input, values others; no rotation.  A loud key lies at
    a place of its own, the same row asks for it hundreds of positions on, in a prompt and decoded: who loses it shows it."""
    width, dim, T, page, p = 64, 16, 700, 64, "l0.mix.left."
    eye = torch.eye(dim, width)
    W = {p + "q": torch.cat([eye] * 2), p + "k": eye, p + "v": torch.cat([torch.zeros(dim, dim), torch.eye(dim, width - dim)], 1),
         p + "o": torch.randn(width, 2 * dim, generator=torch.Generator().manual_seed(3)).to(torch.bfloat16).float()}
    if kind == "normed":
        cfg = config(width, 16, [layer(parallel(heads(2, 1, dim, dim, 1.5), [0.5], 4, 4), None)])
        W.update({p + s + ".b": torch.zeros(n) for s, n in (("q", 2 * dim), ("k", dim), ("v", dim), ("o", width))})
        c = cfg["layers"][0]["mixer"]["left"]
        plain = lambda h: P.turned_normed_attention(doubles(W), p, c, h.double(), 1e-5).float()
    else:
        cfg = config(width, 16, [layer(parallel_2(heads(2, 1, dim, dim, 1.0), 3, 1, 1, 4, 4, 1), None)])
        W.update({p + s + ".conv": torch.tensor([[0.125, 0.25, 1.0]]).repeat(n, 1) for s, n in (("q", 2 * dim), ("k", dim), ("v", dim))})
        W[p + "g"] = torch.zeros(2 * dim, width)
        c = cfg["layers"][0]["mixer"]["left"]
        plain = lambda h: P.convolved_attention(doubles(W), p, c, h.double()).float()
    base = rows_in(T, width, 17, dtype)
    base[:, :dim] *= 0.5
    for at in (0, 63, 64, 200):
        asks = [i for i in (at + 2, 256, 640, 690) if i > at + 1]
        h = base.clone()
        for i in (at, *asks):
            h[i, :dim] = base[at, :dim] * 6.0
        lost = h.clone()
        lost[at, dim:] += 3.0                                  # the key's values changed: who sees it must show it
        if dtype == "bfloat16":
            h, lost = h.to(torch.bfloat16).float(), lost.to(torch.bfloat16).float()
        ref, moved = plain(h), plain(lost)
        for i in asks:
            assert float((moved - ref)[i].abs().max()) > 0.05 * float(ref.abs().max()), (at, i)
        for cuts in ([T], [638, 2] + [1] * 60, [2, 147, 1, 1, 64, 400, 60, 5] + [1] * 20):
            for rows, want in ((h, ref), (lost, moved)):
                part = mixer_of(cfg, "left")
                got = run_mixer(part, W, harness_for(part, dtype, page, T), rows, cuts, width)
                assert float((got - want).abs().max()) <= part_tol(dtype, want), (at, cuts[:4])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("chunk,page", [(12, 8), (100, 64), (64, 64), (65, 64)])
def test_keys_at_the_edges_of_chunks_decide_a_row(chunk, page, dtype):
    """A loud key at a chunk's last place and at the next one's first, asked for from both sides of the edge: seen within its
    chunk only.  Both maps read different places of the input."""
    width, dim, T, p = 64, 16, 400, "l0.mix."
    cfg = config(width, 16, [layer(diff_att(2, 1, dim, dim, chunk=chunk, scale=1.0), None)])
    c = cfg["layers"][0]["mixer"]
    first, second = torch.eye(dim, width), torch.cat([torch.zeros(dim, 48), torch.eye(dim)], 1)
    W = {p + "q": torch.cat([first, second] * 2), p + "k": torch.cat([first, second]),
         p + "v": torch.cat([torch.zeros(dim, dim), torch.eye(dim, width - dim)], 1), p + "g": torch.zeros(2 * dim, width),
         p + "o": torch.randn(width, 2 * dim, generator=torch.Generator().manual_seed(3)).to(torch.bfloat16).float()}
    W.update({p + s + ".b": torch.zeros(n) for s, n in (("q", 4 * dim), ("k", 2 * dim), ("v", dim))})
    W.update({p + s: torch.full((dim,), 0.25) for s in ("lq1", "lk1", "lq2", "lk2")})
    plain = lambda h: P.differential_attention(doubles(W), p, c, h.double(), 1e-5).float()
    base = rows_in(T, width, 18, dtype)
    base[:, :dim] *= 0.5
    edge = (T // 2) // chunk * chunk
    for at in (edge - 1, edge, 0):
        asks = sorted({at + 1, edge - 1, edge, edge + 1, edge + chunk - 1, edge + chunk} - set(range(at + 1)))
        h = base.clone()
        for i in (at, *asks):
            h[i, :dim] = base[at, :dim] * 6.0
        lost = h.clone()
        lost[at, dim:dim + 16] += 3.0
        if dtype == "bfloat16":
            h, lost = h.to(torch.bfloat16).float(), lost.to(torch.bfloat16).float()
        ref, moved = plain(h), plain(lost)
        for i in asks:
            assert (float((moved - ref)[i].abs().max()) > 0.02 * float(ref.abs().max())) == (i // chunk == at // chunk), (at, i)
        for cuts in ([T], [edge - 2] + [1] * 6 + [T - edge - 4], [2, 1, 1, 3] + [1] * 30 + [64, 2, T - 103], [edge + chunk - 2, 2, T - edge - chunk]):
            for rows, want in ((h, ref), (lost, moved)):
                part = mixer_of(cfg)
                got = run_mixer(part, W, harness_for(part, dtype, page, T), rows, cuts, width)
                assert float((got - want).abs().max()) <= part_tol(dtype, want), (at, cuts[:4])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["parallel", "parallel_2"])
def test_pairs_of_mixers_stored_apart_or_added_into_the_stream(kind, dtype):
    """A pair inside a block that only knows `forward`: its sum is added into what is there."""
    width, T = 64, 90
    left = heads(4, 2, 16, 32, **rot(8, 100.0))
    cfg = config(width, 16, [layer(parallel(left, [0.9, 0.5], 16, 16, (0.6, 1.3)) if kind == "parallel" else parallel_2(left, 3, 2, 1, 32, 16, 4), None)])
    W = weights_of(cfg, 47)
    L = cfg["layers"][0]
    plain = lambda W, h: P.mixer(doubles(W), "l0.mix.", L, h.double(), 1e-5)
    check_mixer(cfg, W, plain, dtype, T, [[T], [40] + [1] * 9 + [2, 39]], ranks={"l0.mix.right.a1": 16, "l0.mix.right.g1": 16} if kind == "parallel_2" else None,
                accumulate=True)


# --------------------------------------------------------------------------- passes over the stream
class Slots:
    """Requests in slots with their positions, cut into steps; the device's view of each step."""

    def __init__(self, lengths):
        self.at = [0] * len(lengths)

    def step(self, portions):
        """portions: [(slot, tokens)] -> positions and slots of the step's tokens."""
        pos, rows = [], []
        for slot, n in portions:
            pos += range(self.at[slot], self.at[slot] + n)
            rows += [slot] * n
            self.at[slot] += n
        put = lambda v: torch.tensor(v, dtype=torch.int32).cuda()
        return put(pos), put(rows)


STEPS = [[(2, 1), (0, 5)], [(1, 2), (2, 2), (0, 1)], [(0, 1), (1, 1), (2, 1)], [(2, 6), (1, 3)], [(1, 1), (0, 4)], [(0, 2), (2, 1), (1, 4)],
         [(0, 1)], [(1, 700), (0, 350)]]
LENGTHS = [sum(n for step in STEPS for s, n in step if s == slot) for slot in range(3)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [32, 33, 5000])
@pytest.mark.parametrize("buckets,mul_prev,mul_cur", [(13, 5, 3), (1, 1, 1), (1021, (1 << 31) - 1, 77), (64, 0, 9)])
def test_token_pairs_across_steps(width, buckets, mul_prev, mul_cur, dtype):
    rt = Runtime(dtype)
    g = torch.Generator().manual_seed(1)
    vocab = 50 if width != 32 else 50000
    embed, pairs = (torch.randn(n, width, generator=g).to(torch.bfloat16).float() for n in (vocab, buckets + 1))
    seqs = [torch.randint(0, vocab, (n,), generator=g).tolist() for n in LENGTHS]
    cfg = {"embedding": {"scale": 0.75, "bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}}}
    want = [P.embedding_rows(cfg, {"embed": embed.double(), "bigram": pairs.double()}, s).float() for s in seqs]
    slots, state = Slots(LENGTHS), torch.full((4, 2), 12345, dtype=torch.int32, device="cuda")
    for step in STEPS:
        before = list(slots.at)
        pos, rows = slots.step(step)
        toks = [t for s, n in step for t in seqs[s][before[s]:before[s] + n]]
        out = torch.empty(len(toks), width, device="cuda")
        again = 2 if all(n == 1 for _, n in step) else 1           # a step of single tokens may be run again
        for _ in range(again):
            rt.k.embed_pairs(torch.tensor(toks, dtype=torch.int32).cuda(), embed.to(rt.dtype).cuda(), 0.75, pairs.to(rt.dtype).cuda(), mul_prev,
                             mul_cur, state, pos, rows, out)
            ref = torch.cat([want[s][before[s]:before[s] + n] for s, n in step])
            assert float((out.cpu() - ref).abs().max()) <= 2e-6 * float(ref.abs().max())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [64, 33, 130, 4608])
def test_a_token_shift_across_steps(width, dtype):
    """Norm and shift in steps of any portions, and in steps of single tokens as part of the pass that sums (equal bits)."""
    rt = Runtime(dtype)
    g = torch.Generator().manual_seed(2)
    eps, w, share = 1e-4, torch.randn(width, generator=g) * 0.3, torch.rand(width, generator=g)
    xs = [torch.randn(n, width, generator=g) * 2 for n in LENGTHS]
    want = [P.shifted(P.around_zero_norm({"n": w.double()}, "n", x.double(), eps), share.double()) for x in xs]
    gain = (1.0 + w).cuda()
    slots, state = Slots(LENGTHS), torch.zeros(4, 2 * width, device="cuda")
    tol = 2e-6 if dtype == "float32" else 1e-2
    for step in STEPS:
        before = list(slots.at)
        pos, rows = slots.step(step)
        x = torch.cat([xs[s][before[s]:before[s] + n] for s, n in step]).cuda()
        ref = torch.cat([want[s][before[s]:before[s] + n] for s, n in step])
        out = torch.empty(len(x), width, dtype=rt.dtype, device="cuda")
        was = state.clone()
        rt.k.shifted_norm(x, gain, eps, share.cuda(), state, pos, rows, out)
        assert float((out.cpu().double() - ref).abs().max()) <= tol * max(1.0, float(ref.abs().max()))
        if all(n == 1 for _, n in step):
            y, s = torch.randn(len(x), width, generator=g).cuda(), torch.ones(width).cuda()
            base, out2, other = x - y, torch.empty_like(out), was.clone()
            for again in range(2):
                total = base.clone()
                rt.k.scaled_sum([(y, s, None)], total, norm=(gain, eps, out2), shift=(share.cuda(), other, pos, rows))
                assert float((out2.cpu().double() - ref).abs().max()) <= tol * max(1.0, float(ref.abs().max())) * (4 if dtype == "float32" else 1)
            exact = was.clone()
            rt.k.shifted_norm(total, gain, eps, share.cuda(), exact, pos, rows, out)
            assert torch.equal(out, out2) and torch.equal(exact, other)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width", [(1, 64), (5, 33), (7, 2048), (300, 130), (3, 4612)])
def test_a_scaled_sum_with_norms(rows, width, dtype):
    rt = Runtime(dtype)
    g = torch.Generator().manual_seed(rows)
    x, y0, y1 = (torch.randn(rows, width, generator=g) * 2 for _ in range(3))
    s0, s1, w = (torch.randn(width, generator=g) for _ in range(3))
    tol = 3e-6 if dtype == "float32" else 1e-2
    for eps0, eps1 in ((None, None), (0.1, 1e-5), (None, 1e-3)):
        for two in (False, True):
            n = lambda y, eps: y.double() if eps is None else P.unit(y.double(), eps)
            want = x.double() + n(y0, eps0) * s0.double() + (n(y1, eps1) * s1.double() if two else 0.0)
            got, h = x.cuda().clone(), torch.empty(rows, width, dtype=rt.dtype, device="cuda")
            terms = [(y0.cuda(), s0.cuda(), eps0)] + ([(y1.cuda(), s1.cuda(), eps1)] if two else [])
            rt.k.scaled_sum(terms, got, norm=((1.0 + w).cuda(), 1e-4, h))
            assert float((got.cpu().double() - want).abs().max()) <= 3e-6 * float(want.abs().max())
            ref = P.around_zero_norm({"n": w.double()}, "n", want, 1e-4)
            assert float((h.cpu().double() - ref).abs().max()) <= tol * max(1.0, float(ref.abs().max()))
            plain = x.cuda().clone()
            rt.k.scaled_sum(terms, plain)
            assert torch.equal(plain, got)


def test_wrong_shapes_are_refused():
    rt = Runtime("float32")
    z = lambda *s: torch.zeros(*s, device="cuda")
    i = lambda *s: torch.zeros(*s, dtype=torch.int32, device="cuda")
    with pytest.raises(KernelError):
        rt.k.shifted_norm(z(2, 8), z(8), 1e-5, z(8), z(1, 8), i(2), i(2), z(2, 8))               # a state of one row
    with pytest.raises(KernelError):
        rt.k.scaled_sum([(z(2, 8), z(7), None)], z(2, 8))
    with pytest.raises(KernelError):
        rt.k.lightning_scan(z(2, 24), 0, 8, 16, True, z(2), z(1, 64), 32, None, i(2), i(2), z(2, 8), 2, 8, 4)    # keys beyond the rows
    with pytest.raises(KernelError):
        rt.k.embed_pairs(i(2), z(4, 8), 1.0, z(1, 8), 1, 1, i(1, 2), i(2), i(2), z(2, 8))        # no bucket
    with pytest.raises(KernelError):
        rt.k.heads_prepare(z(2, 24), 0, 1, 8, 1, 16, 8, 8, None, None, 0.0, 0, False, 1.0, z(2, 0, 2), i(2), i(2), i(1, 1),
                           z(1, 1, 8, 16), 8, z(2, 8), conv=(z(24, 3), z(1, 64), 32, None))      # a state too small for two rows of 24, twice
    build_part("mixer", PartSpec("lightning_attention", dict(hidden_size=8, heads=1, dim=4, vdim=4, decay=[0.5], eps=1e-5)))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("m,n,k", [(3, 64, 64), (16, 40, 128), (40, 192, 256), (100, 130, 64), (300, 128, 2048), (700, 512, 4096), (33, 17, 30)])
def test_a_product_whose_squared_relu_is_its_epilogue(m, n, k, dtype):
    from axon_amd.kernels import MODE_RELU_SQUARED, MODE_STORE_F32
    rt = Runtime(dtype)
    g = torch.Generator().manual_seed(m)
    x, w = torch.randn(m, k, generator=g).to(rt.dtype).cuda(), (torch.randn(n, k, generator=g) * k ** -0.5).to(rt.dtype).cuda()
    for matrix in (rt.k.prepare_weight(w), w):
        got = rt.k.gemm(x, matrix, torch.empty(m, n, dtype=rt.dtype, device="cuda"), None, MODE_RELU_SQUARED)
        sums = rt.k.gemm(x, matrix, torch.empty(m, n, device="cuda"), None, MODE_STORE_F32)
        assert torch.equal(got, (torch.relu(sums) ** 2).to(rt.dtype))          # of the unrounded sums, rounded once
    want = torch.relu(x.double() @ w.double().T) ** 2
    assert float((got.double() - want).abs().max()) <= (2e-5 if dtype == "float32" else 2e-2) * float(want.abs().max())
