"""The Lilunex decoder through the engine against the plain implementation (tests/plain/lilunex_plain.py): whole
prompts, decoding token by token from the first token on, portions down to two tokens, unequal requests side by side
with pages and slots that come round again, long stretches and long decoding, generation through the engine's own entry
point (with pages running out as well), the command line, the trace replay program, and every mechanism alone with
weights or inputs made so that a fault shows (a kept position or a sink left out, a window one position off, a far key
lost, a state not carried across a cut, a correction in the weights: each differs from the plain implementation by far
more than the tolerance)."""
import math
import os
import subprocess
import sys

import pytest
import torch

import axon_amd
from axon_amd.config import config_from_dict
from axon_amd.engine import StepEntry
from axon_amd.parts import CacheBinding, build_part
from axon_amd.weights import WeightStore
from gpu_helpers import DTYPES, DictSource, PartHarness
from helpers import ROOT, TraceBuilder, engine_for, run_trace, tolerance
from lilunex_models import MODELS, att, config, delta, draw_weights, layer, make, moe, wkv
from plain import lilunex_plain as P

pytestmark = pytest.mark.gpu

SLACK = 0.05          # how far 16 bits of stream may move a router's score


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            made[name] = make(str(tmp_path_factory.mktemp("lilunex_" + name)), name)
        return made[name]
    return get


@pytest.fixture(scope="module")
def plain_logits(folders):
    """The plain implementation's logits of a model's test sequences.  float32: its own choice of experts.
    bfloat16: with the experts the engine chose where these are a close call of its own choice (16 bits
    decide a close call either way, and every later row sees it)."""
    kept, models = {}, {}

    def get(name, seq, dtype="float32", forced=None):
        if name not in models:
            models[name] = P.load_plain(folders(name))
        cfg, W = models[name]
        if dtype == "bfloat16":
            return P.forward_logits(cfg, W, seq, forced, SLACK).float()
        key = (name, tuple(seq))
        if key not in kept:
            kept[key] = P.forward_logits(cfg, W, seq).float()
        return kept[key]
    return get


def sequences(name, lengths, seed=0):
    g = torch.Generator().manual_seed(seed)
    return [torch.randint(0, MODELS[name]["cfg"]["vocab"], (n,), generator=g).tolist() for n in lengths]


def assert_close(got, ref, dtype, what):
    """Rows of logits against the plain implementation's.  32-bit: every row within rounding.  16 bits: a head's
    output is divided by its root mean square, and a row whose output happens to be small passes its rounding on many
    times enlarged; so one row in a hundred may reach twice the limit of the others."""
    err = (got - ref).abs().max(dim=-1).values
    limit = tolerance(dtype, ref) * (2.0 if dtype == "float32" else 3.0)
    if dtype == "float32":
        assert float(err.max()) <= limit, f"{what}: {float(err.max())} > {limit} at row {int(err.argmax())}"
        return
    over = int((err > limit).sum())
    assert over <= max(1, len(err) // 100) and float(err.max()) <= 2 * limit, \
        f"{what}: {over} of {len(err)} rows over {limit}, the worst {float(err.max())} at row {int(err.argmax())}"


class RouterLog:
    """What the engine's router chose, launch by launch: the kernels' entry is wrapped while a schedule runs."""

    def __init__(self, k):
        self.k, self.calls = k, []

    def __enter__(self):
        inner = self.k.route_scored

        def logged(logits, correction, top, groups, keep, scale, chosen, weights, **kw):
            inner(logits, correction, top, groups, keep, scale, chosen, weights, **kw)
            self.calls.append(chosen.cpu().tolist())
        self.k.route_scored = logged
        return self

    def __exit__(self, *exc):
        del self.k.route_scored


def run_schedule(eng, name, seqs, schedule):
    """schedule: steps of [(request, tokens)]; every position's logits are asked for.  A request ends with
    its last token.  Returns ({request: [len, vocab]}, {request: {layer: chosen experts by position}})."""
    cfg = MODELS[name]["cfg"] if isinstance(name, str) else name
    routed = [i for i, L in enumerate(cfg["layers"]) if L.get("mlp") and L["mlp"]["kind"] == "moe"]
    at = {r: 0 for r in seqs}
    got = {r: [] for r in seqs}
    chose = {r: {i: [] for i in routed} for r in seqs}
    with RouterLog(eng.rt.k) as log:
        for step in schedule:
            entries, ends = [], []
            for rid, n in step:
                toks = seqs[rid][at[rid]:at[rid] + n]
                entries.append(StepEntry(rid, toks, list(range(len(toks)))))
                at[rid] += len(toks)
                if at[rid] == len(seqs[rid]):
                    ends.append(rid)
            del log.calls[:]
            out = eng.step(entries, ends).cpu()
            assert len(log.calls) == len(routed)
            row = 0
            for e in entries:
                got[e.id].append(out[row:row + len(e.tokens)].clone())
                for i, call in zip(routed, log.calls):
                    chose[e.id][i] += call[row:row + len(e.tokens)]
                row += len(e.tokens)
    assert all(at[r] == len(seqs[r]) for r in seqs)
    return {r: torch.cat(v) for r, v in got.items()}, chose


def pages_for(name, tokens):
    return -(-tokens // MODELS[name]["page"]) + 2


# --------------------------------------------------------------------------- whole models
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MODELS))
def test_whole_prompts_and_decoding_token_by_token(folders, plain_logits, name, dtype):
    n = 200 if name == "B" else 90
    (seq,) = sequences(name, [n], seed=1)
    eng = engine_for(folders(name), dtype, MODELS[name]["page"], pages_for(name, n), max_seqs=2, max_seq_len=256)
    got, chose = run_schedule(eng, name, {"a": seq}, [[("a", n)]])
    ref = plain_logits(name, seq, dtype, chose["a"])
    whole = got["a"]
    assert_close(whole, ref, dtype, "whole prompt")
    # from the first token on, one token a step: the first tokens of a sequence (a state, a shift and a convolution
    # that start from nothing), every page's edge, every window's edge
    got, chose = run_schedule(eng, name, {"b": seq}, [[("b", 1)] for _ in range(n)])
    single = got["b"]
    assert_close(single, plain_logits(name, seq, dtype, chose["b"]), dtype, "token by token")
    # most of it at once, the rest decoded
    got, chose = run_schedule(eng, name, {"c": seq}, [[("c", n - 45)]] + [[("c", 1)] for _ in range(45)])
    assert_close(got["c"], plain_logits(name, seq, dtype, chose["c"]), dtype, "prompt then decoding")
    if dtype == "float32":
        assert float((single - whole).abs().max()) <= 2 * tolerance(dtype, ref)
    eng.cache.check()


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
        got, chose = run_schedule(eng, name, {"a": seq}, sched)
        assert_close(got["a"], plain_logits(name, seq, dtype, chose["a"]), dtype, f"portions {cuts}")
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
    got, chose = run_schedule(eng, name, seqs, sched)
    for r in seqs:
        assert_close(got[r], plain_logits(name, seqs[r], dtype, chose[r]), dtype, f"request {r} in the mixed schedule")
    eng.cache.check()
    assert not eng.live
    for g in range(len(eng.cache.groups)):
        assert eng.cache.free_pages(g) == eng.cache.groups[g].n_pages
    if dtype == "float32":
        # each request alone gives the same rows as side by side, to rounding
        alone, _ = run_schedule(eng, name, {2: seqs[2]}, [[(2, lengths[2])]])
        assert float((alone[2] - got[2]).abs().max()) <= 2 * tolerance(dtype, plain_logits(name, seqs[2]))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B", "C", "E"])
def test_long_stretches_run_the_scans_in_segments(folders, plain_logits, name, dtype):
    """Hundreds of tokens of a request in one step: the scans cut the stretch into pieces that run side by side; the
    state they leave is what later portions and decoded tokens go on from.  Beside a short request in the same step."""
    n = 720
    long, short = sequences(name, [n, 9], seed=5)
    page = MODELS[name]["page"]
    eng = engine_for(folders(name), dtype, page, -(-n // page) + 4, max_seqs=2, max_seq_len=768, max_batch_tokens=544)
    seen = []
    inner = eng.rt.k.wkv_scan

    def logged(*a, segments=None, **kw):
        seen.append(None if segments is None else segments[0].shape[0])
        return inner(*a, segments=segments, **kw)
    eng.rt.k.wkv_scan = logged
    try:
        got, chose = run_schedule(eng, name, {"a": long, "b": short}, [[("a", 530), ("b", 4)], [("a", 1), ("b", 5)], [("a", 2)], [("a", 187)]])
    finally:
        del eng.rt.k.wkv_scan
    assert any(k is not None and k > 2 for k in seen) and any(k is None for k in seen)
    assert_close(got["a"], plain_logits(name, long, dtype, chose["a"]), dtype, "the long request")
    assert_close(got["b"], plain_logits(name, short, dtype, chose["b"]), dtype, "the short request beside it")
    eng.cache.check()


@pytest.mark.parametrize("name", ["A", "C", "D"])
def test_long_decoding_across_many_pages(folders, plain_logits, name):
    n = 250
    (seq,) = sequences(name, [n], seed=4)
    ref = plain_logits(name, seq)
    eng = engine_for(folders(name), "float32", MODELS[name]["page"], pages_for(name, n), max_seqs=1, max_seq_len=256)
    got, _ = run_schedule(eng, name, {"a": seq}, [[("a", 3)]] + [[("a", 1)] for _ in range(n - 3)])
    assert_close(got["a"], ref, "float32", "long decoding")


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
            assert float(row.max() - row[tok]) <= 0.3 * tolerance("bfloat16", logits)


@pytest.mark.parametrize("name", ["A", "D"])
def test_generation_goes_on_where_pages_run_out(folders, name):
    """A pool that three requests outgrow while they generate: the youngest gives up its pages (those of its kept first
    positions among them) and its state, and is fed again later; the tokens are those of a roomy pool."""
    page = MODELS[name]["page"]
    prompts = sequences(name, [2 * page, 2 * page - 3, page + 1], seed=8)
    load = lambda pages: axon_amd.load(folders(name), dtype="float32", page_size=page, num_pages=pages, max_seqs=3, max_seq_len=128)
    want = load(64).generate(prompts, max_new_tokens=40)
    tight = load(-(-(2 * page + 40) // page) + 3)
    assert tight.generate(prompts, max_new_tokens=40) == want
    assert tight.last_stats.preemptions > 0
    tight.engine.cache.check()


def test_the_command_line_generates_with_the_design(folders):
    name = "C"
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
    name = "E"                     # (without routers that see pages: no close call of an expert between the runs)
    seqs = sequences(name, [40, 17, 64], seed=7)
    refs = [plain_logits(name, s) for s in seqs]
    tb = TraceBuilder()
    tb.step([("a", seqs[0][:30], [0, 29]), ("b", seqs[1][:2], [1])])
    tb.step([("a", seqs[0][30:31], [0]), ("b", seqs[1][2:], [0, 14]), ("c", seqs[2][:7], [])], end=["b"])
    tb.step([("a", seqs[0][31:], [8]), ("c", seqs[2][7:], [0, 56])], end=["a", "c"])
    rows = tb.collect(run_trace(folders(name), dtype, tb.steps, str(tmp_path), max_tokens=192))
    for (rid, pos), row in rows.items():
        ref = refs["abc".index(rid)]
        assert float((torch.from_numpy(row) - ref[pos]).abs().max()) <= (3 if dtype == "float32" else 5) * tolerance(dtype, ref)


# --------------------------------------------------------------------------- the mechanisms alone
def rows_in(T, width, seed, dtype, scale=1.0):
    """Random rows; for the 16-bit run, rows that 16 bits hold exactly (the plain run starts from the same numbers)."""
    g = torch.Generator().manual_seed(seed)
    h = torch.randn(T, width, generator=g) * scale
    return h.to(torch.bfloat16).float() if dtype == "bfloat16" else h


def part_tol(dtype, ref):
    return (3e-5 if dtype == "float32" else 3e-2) * max(1.0, float(ref.abs().max()))


def one_layer(width, mixer, mlp=None, eps=1e-5):
    return config(width, 16, [layer(mixer, mlp)], eps=eps)


def mixer_of(cfg, rank=None, index=0):
    c = config_from_dict(cfg)
    if rank is not None:
        c = c.with_sizes({f"l{index}.mix.w1": (rank, cfg["width"])})
    return build_part("mixer", c.layers[index]["mixer"], f"l{index}.")


def run_mixer(part, harness, h, cuts, width):
    """The mixer's 32-bit output for rows h, fed in portions of the given sizes."""
    outs, at = [], 0
    for n in cuts:
        ctx = harness.ctx([0] * n)
        x = h[at:at + n].to(harness.rt.dtype).cuda()
        out = torch.full((n, width), float("nan"), dtype=torch.float32, device="cuda")
        part.forward(ctx, CacheBinding(group=0, index=0, writes=True, state_index=0), x, out, accumulate=False)
        outs.append(out.cpu())
        at += n
    assert at == h.shape[0]
    return torch.cat(outs)


def loaded(part, W, harness):
    part.load(WeightStore(DictSource(W), harness.rt.device, harness.rt.dtype), harness.rt)
    return part


CUTS = lambda T, page: [[T], [page - 1] + [1] * 8 + [T - page - 7], [2, 1, 1, 3] + [1] * 30 + [64, 2, T - 103], [1] * T]


def check_state_mixer(cfg, W, plain, dtype, T, cut_sets, rank=None, h=None, rows=slice(None), max_seq_len=256):
    h = rows_in(T, cfg["width"], 13, dtype) if h is None else h
    ref = plain(W, h).float()
    for cuts in cut_sets:
        part = mixer_of(cfg, rank)
        ss = part.state_spec()
        hs = PartHarness(dtype, None, state_elems=[(ss.elems, ss.dtype)], max_seq_len=max_seq_len)
        got = run_mixer(loaded(part, W, hs), hs, h, cuts, cfg["width"])
        err = (got - ref)[rows].abs().max(dim=-1).values
        # 16 bits: a row whose head happens to come out small passes its rounding on enlarged
        assert float(err.max()) <= part_tol(dtype, ref) * (1 if dtype == "float32" else 3), (cuts[:8], float(err.max()), int(err.argmax()))
        assert float(err.median()) <= part_tol(dtype, ref), (cuts[:8], float(err.median()))
    return h, ref


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dim,rank,width", [(3, 5, 3, 42), (4, 32, 64, 64), (2, 70, 16, 48), (1, 40, 1, 80), (8, 64, 80, 64),
                                                  (2, 130, 33, 64), (1, 256, 16, 64), (5, 12, 7, 33)])
def test_time_mixing_alone_in_portions(heads, dim, rank, width, dtype):
    """The walk with its state and the row before carried across cuts of every kind: whole, a token at a time from the
    first token on, portions down to one token.  Decays from a step to hundreds of steps."""
    T = 140
    cfg = one_layer(width, wkv(heads, dim), eps=1e-3)
    W = {k: v for k, v in draw_weights(cfg, 41, {0: rank}).items() if k.startswith("l0.mix.")}
    c = cfg["layers"][0]["mixer"]
    plain = lambda W, h: P.wkv_mixer({k: v.double() for k, v in W.items()}, "l0.mix.", c, h.double(), 1e-3)
    h, ref = check_state_mixer(cfg, W, plain, dtype, T, CUTS(T, 16), rank)
    # what the test would catch: a state or a shift that starts anew at a cut, the bonus left out, the gate, w0
    loud = 20 * part_tol("float32", ref)
    anew = torch.cat([plain(W, h[:100]), plain(W, h[100:])]).float()
    assert float((anew - ref)[108:].abs().max()) > loud
    Wd = {k: v.double() for k, v in W.items()}
    shift = P.shifted
    try:
        P.shifted = lambda x: torch.cat([x[:1], shift(x)[1:]])           # the first token's shift reads itself, not zeros
        assert float((plain(W, h).float() - ref)[0].abs().max()) > loud
    finally:
        P.shifted = shift
    for name in ("u", "w0", "mu.w", "mu.g"):
        other = dict(Wd, **{"l0.mix." + name: torch.zeros_like(Wd["l0.mix." + name])})
        assert float((plain(other, h).float() - ref).abs().max()) > loud, name


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,conv", [(3, 1, 5, 7, 3), (4, 2, 64, 32, 4), (2, 2, 132, 24, 1), (1, 1, 16, 40, 5),
                                                          (6, 3, 200, 16, 2), (8, 4, 128, 128, 4), (2, 1, 32, 72, 4), (4, 4, 6, 9, 2),
                                                          (3, 3, 96, 80, 3), (6, 2, 32, 16, 2)])
def test_the_delta_rule_alone_in_portions(heads, kv_heads, dim, vdim, conv, dtype):
    """The walk with its state and the convolutions' kept inputs carried across cuts of every kind: whole, a token at a
    time from the first token on, portions that end inside the convolutions' reach."""
    width, T = 48, 140
    cfg = one_layer(width, delta(heads, kv_heads, dim, vdim, conv), eps=1e-3)
    W = {k: v for k, v in draw_weights(cfg, 43).items() if k.startswith("l0.mix.")}
    c = cfg["layers"][0]["mixer"]
    plain = lambda W, h: P.delta_mixer({k: v.double() for k, v in W.items()}, "l0.mix.", c, h.double(), 1e-3)
    h, ref = check_state_mixer(cfg, W, plain, dtype, T, CUTS(T, 16))
    loud = 20 * part_tol("float32", ref)
    anew = torch.cat([plain(W, h[:100]), plain(W, h[100:])]).float()
    assert float((anew - ref)[108:].abs().max()) > loud
    # read before the token's write, no correction along the key, keys that are not of length 1, the decay behind the read
    rule = P.delta_recurrence
    try:
        P.delta_recurrence = lambda q, k, v, g, beta: rule(q, k, v, torch.ones_like(g), beta)
        assert float((plain(W, h).float() - ref).abs().max()) > loud
        P.delta_recurrence = lambda q, k, v, g, beta: torch.cat([torch.zeros_like(v[:1]), rule(q[1:].clone(), k[:-1], v[:-1], g[:-1], beta[:-1])])
        assert float((plain(W, h).float() - ref).abs().max()) > loud
    finally:
        P.delta_recurrence = rule
    length = P.unit_length
    try:
        P.unit_length = lambda x: x
        assert float((plain(W, h).float() - ref).abs().max()) > loud
    finally:
        P.unit_length = length


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["wkv", "delta"])
def test_a_slow_state_remembers_an_input_hundreds_of_positions_back(kind, dtype):
    """Decays set by hand to 0.999 a step, a loud row at position 3 and faint rows after it: 600 positions on, the output
    is still that row's doing, in a prompt and decoded one token at a time."""
    width, T = 32, 640
    if kind == "wkv":
        cfg = one_layer(width, wkv(1, 16), eps=1e-3)
        W = {k: v for k, v in draw_weights(cfg, 43, {0: 16}).items() if k.startswith("l0.mix.")}
        W["l0.mix.w0"] = torch.full_like(W["l0.mix.w0"], math.log(0.001))
        W["l0.mix.w2"] = torch.zeros_like(W["l0.mix.w2"])
        plain = lambda W, h: P.wkv_mixer({k: v.double() for k, v in W.items()}, "l0.mix.", cfg["layers"][0]["mixer"], h.double(), 1e-3)
        rank = 16
    else:
        cfg = one_layer(width, delta(1, 1, 64, 8, 2), eps=1e-3)
        W = {k: v for k, v in draw_weights(cfg, 43).items() if k.startswith("l0.mix.")}
        W["l0.mix.A_log"] = torch.tensor([math.log(0.001)])
        W["l0.mix.dt_bias"] = torch.tensor([0.5413])                # softplus gives 1: g = exp(-0.001)
        W["l0.mix.a"] = torch.zeros_like(W["l0.mix.a"])
        # the loud row writes, the faint ones read: a logit of beta that the loud row alone lifts
        W["l0.mix.b"] = torch.zeros_like(W["l0.mix.b"])
        W["l0.mix.b"][0, 0] = 4.0
        plain = lambda W, h: P.delta_mixer({k: v.double() for k, v in W.items()}, "l0.mix.", cfg["layers"][0]["mixer"], h.double(), 1e-3)
        rank = None
    W = {k: v.to(torch.bfloat16).float() for k, v in W.items()}
    h = rows_in(T, width, 15, dtype, scale=0.02 if kind == "wkv" else 1.0)
    h[3] = rows_in(1, width, 16, dtype, scale=3.0)[0]
    if kind == "delta":
        h[:, 0] = -3.0
        h[3, 0] = 3.0
    ref = plain(W, h).float()
    quiet = h.clone()
    quiet[3] = h[4]
    assert float((plain(W, quiet).float() - ref)[600:].abs().max()) > 0.2 * float(ref[600:].abs().max())
    check_state_mixer(cfg, W, plain, dtype, T, ([T], [600] + [1] * 40, [2, 3, 64, 129, 1, 1, 400, 38, 2]), rank, h, slice(600, None), 1024)


def check_attention(cfg, W, plain, page, dtype, T, cut_sets, h=None, rows=slice(None), index=0):
    h = rows_in(T, cfg["width"], 13, dtype) if h is None else h
    ref = plain(W, h).float()
    for cuts in cut_sets:
        part = mixer_of(cfg)
        hs = PartHarness(dtype, part.cache_spec(), page_size=page, n_pages=-(-T // page) + 3, max_seq_len=1024)
        got = run_mixer(loaded(part, W, hs), hs, h, cuts, cfg["width"])
        assert float((got - ref)[rows].abs().max()) <= part_tol(dtype, ref), (cuts[:8], int((got - ref).abs().max(dim=-1).values.argmax()))
    return h, ref


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,mask,rot,page", [
    (3, 1, 10, 6, (7, 3), (4, 100.0, 2.0), 8), (8, 2, 32, 32, (70, 4), (32, 100.0, 4.0), 64), (4, 4, 64, 48, (1, 1), (32, 100.0, None), 64),
    (1, 1, 24, 40, (5, 30), None, 16), (6, 3, 48, 16, (128, 65), (48, 100.0, 8.0), 128), (8, 2, 128, 128, (64, 1), (64, 100.0, 2.0), 64),
    (32, 2, 64, 64, (63, 64), (64, 100.0, 2.0), 64), (4, 1, 256, 192, (33, 130), (128, 100.0, 2.0), 64),
    (8, 8, 96, 80, (40, 5), (96, 50.0, 3.0), 64), (4, 2, 32, 32, None, (32, 100.0, 4.0), 64), (16, 16, 16, 272, (20, 7), (16, 9.0, 2.0), 64)])
def test_attention_with_a_window_beside_kept_positions(heads, kv_heads, dim, vdim, mask, rot, page, dtype):
    cfg = one_layer(64, att(heads, kv_heads, dim, vdim, mask=mask, rot=rot))
    W = {k: v for k, v in draw_weights(cfg, 31).items() if k.startswith("l0.mix.")}
    c = cfg["layers"][0]["mixer"]
    plain = lambda W, h, c=c: P.attention_mixer({k: v.double() for k, v in W.items()}, "l0.mix.", c, h.double(), 1e-5)
    T = 200
    h, ref = check_attention(cfg, W, plain, page, dtype, T, CUTS(T, page)[:3] + [[60] + [1] * 10 + [56] + [1] * 74])
    # what the test would catch: windows and kept positions one off, sinks, biases and gains left out, norms per head
    loud = 20 * part_tol("float32", ref)
    wrong = lambda **kw: float((plain(W, h, dict(c, **kw)).float() - ref).abs().max()) > loud
    if mask is not None:
        size, keep = mask
        assert wrong(mask={"size": size + 1, "keep_first": keep}) and wrong(mask={"size": size, "keep_first": keep + 1})
        assert wrong(mask={"size": size, "keep_first": keep - 1})
    if rot is not None:
        assert wrong(rot=dict(c["rot"], scaling={"factor": 16.0})) and wrong(rot=None)
    for name in ("sink", "q.b", "k.b", "v.b", "o.b", "k.norm"):
        if name == "k.b" and dim == 10:
            continue
        other = dict(W, **{"l0.mix." + name: torch.zeros_like(W["l0.mix." + name]) - (50.0 if name == "sink" else 0.0)})
        assert float((plain(other, h).float() - ref).abs().max()) > loud, name
    if heads > 1:
        unit = P.unit
        try:
            P.unit = lambda x, eps: unit(x.view(*x.shape[:-1], -1, dim), eps).view_as(x)
            assert float((plain(W, h).float() - ref).abs().max()) > loud
        finally:
            P.unit = unit


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,page,size,keep", [(2, 1, 8, 12, 3), (8, 2, 64, 100, 2), (3, 3, 16, 64, 17), (16, 4, 64, 65, 70),
                                                           (4, 4, 64, 300, 1)])
def test_keys_at_every_edge_of_a_window_decide_a_row(heads, kv_heads, page, size, keep, dtype):
    """Weights set by hand: queries and keys read the same places of the input, values others.  A loud key lies at a
    place, and the same loud row asks for it from just inside the window, just outside it, hundreds of positions on, in a
    prompt and decoded: at the last kept position it is seen from everywhere, at the first that is not kept from inside
    the window only."""
    width, dim, T = 64, 16, 700
    cfg = one_layer(width, att(heads, kv_heads, dim, dim, mask=(size, keep), scale=1.5))
    c = cfg["layers"][0]["mixer"]
    g = torch.Generator().manual_seed(3)
    p = "l0.mix."
    W = {p + "q": torch.cat([torch.eye(dim, width)] * heads), p + "k": torch.cat([torch.eye(dim, width)] * kv_heads),
         p + "v": torch.cat([torch.cat([torch.zeros(dim, dim), torch.eye(dim, width - dim)], 1)] * kv_heads),
         p + "q.norm": torch.ones(heads * dim), p + "k.norm": torch.ones(kv_heads * dim), p + "sink": torch.full((heads,), -2.0),
         p + "o": torch.randn(width, heads * dim, generator=g).to(torch.bfloat16).float()}
    for s, n in (("q", heads * dim), ("k", kv_heads * dim), ("v", kv_heads * dim), ("o", width)):
        W[p + s + ".b"] = torch.zeros(n)
    plain = lambda W, h, c=c: P.attention_mixer({k: v.double() for k, v in W.items()}, p, c, h.double(), 1e-5)
    base = rows_in(T, width, 17, dtype)
    key = base[0, :dim].clone()
    for at in (keep - 1, keep, 200):
        asks = sorted({at + size - 1, at + size, at + size + 1, 650, 690} - {at})
        h = base.clone()
        for i in (at, *asks):
            h[i, :dim] = key
        lost = h.clone()
        lost[at, dim:] += 3.0                                  # the key's values changed: who sees it must show it
        if dtype == "bfloat16":
            lost = lost.to(torch.bfloat16).float()
        ref, moved = plain(W, h).float(), plain(W, lost).float()
        for i in asks:
            sees = i - at < size or at < keep
            assert (float((moved - ref)[i].abs().max()) > 0.05 * float(ref.abs().max())) == sees, (at, i)
        edge = at + size - 2
        for cuts in ([T], [edge] + [1] * 5 + [T - edge - 5], [640 - 2, 2] + [1] * 60, [2, 147, 1, 1, 64, 400, 60, 5] + [1] * 20):
            for rows, want in ((h, ref), (lost, moved)):
                part = mixer_of(cfg)
                hs = PartHarness(dtype, part.cache_spec(), page_size=page, n_pages=-(-T // page) + 3, max_seq_len=1024)
                got = run_mixer(loaded(part, W, hs), hs, rows, cuts, width)
                assert float((got - want).abs().max()) <= part_tol(dtype, want), (at, cuts[:4])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("experts,identity,top,ff,shared", [(5, 2, 2, 24, 16), (4, 0, 4, 64, 96), (6, 1, 1, 32, None), (8, 3, 3, 48, 8),
                                                            (40, 8, 6, 32, 64), (2, 6, 5, 16, 8)])
def test_experts_beside_identities(experts, identity, top, ff, shared, dtype):
    width, T = 64, 70
    cfg = one_layer(width, wkv(1, 8), moe(experts, identity, top, ff, shared))
    W = {k: v for k, v in draw_weights(cfg, 35).items() if k.startswith("l0.mlp.")}
    c = cfg["layers"][0]["mlp"]
    for T in (70, 300):                                       # lists in tiles of 16 rows and of 64
        part = build_part("feed_forward", config_from_dict(cfg).layers[0]["mlp"], "l0.")
        hs = PartHarness(dtype, max_seq_len=1024)
        loaded(part, W, hs)
        h = rows_in(T, width, 19, dtype)
        Wd = {k: v.double() for k, v in W.items()}
        with RouterLog(hs.rt.k) as log:
            out = torch.full((T, width), 1.0, dtype=torch.float32, device="cuda")
            part.forward(hs.ctx([0] * T), h.to(hs.rt.dtype).cuda(), out)                    # adds into what is there
            stored = torch.full((T, width), float("nan"), dtype=torch.float32, device="cuda")
            part.forward(hs.ctx([0] * T), h.to(hs.rt.dtype).cuda(), stored, accumulate=False)
        if identity:
            assert any(e >= experts for row in log.calls[0] for e in row)
        ref = P.experts_ff(Wd, "l0.mlp.", c, h.double(), log.calls[0] if dtype == "bfloat16" else None, SLACK).float()
        assert float((stored.cpu() - ref).abs().max()) <= part_tol(dtype, ref)
        assert float((out.cpu() - 1.0 - ref).abs().max()) <= part_tol(dtype, ref)
    # what the test would catch: a correction in the weights or not in the choice, weights not over their sum, the softmax
    # over experts alone, identities that give nothing, the shared expert's gate left out
    h, loud = h[:70].double(), 20 * part_tol("float32", ref)
    ref = ref[:70]
    differs = lambda W, c=c: float((P.experts_ff(W, "l0.mlp.", c, h).float() - ref).abs().max()) > loud
    if top < experts + identity:
        assert differs(dict(Wd, **{"l0.mlp.correction": torch.zeros_like(Wd["l0.mlp.correction"])}))
    scores = P.router_scores
    try:
        P.router_scores = lambda W, p, x: scores(W, p, x) + W[p + "correction"]
        if top > 1:
            assert differs(Wd)
    finally:
        P.router_scores = scores
    if shared:
        assert differs(dict(Wd, **{"l0.mlp.shared.sg": torch.zeros_like(Wd["l0.mlp.shared.sg"])}))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,dim", [(1, 64), (5, 33), (7, 2048), (300, 130), (3, 4100)])
def test_dynamic_tanh_alone_and_with_the_sum_and_the_next_norm(rows, dim, dtype):
    from axon_amd.engine import Runtime
    rt = Runtime(dtype)
    g = torch.Generator().manual_seed(rows)
    x, y = torch.randn(rows, dim, generator=g) * 2, torch.randn(rows, dim, generator=g) * 2
    store = torch.float32 if dtype == "float32" else torch.bfloat16
    norms = [(a, torch.randn(dim, generator=g).to(store), torch.randn(dim, generator=g).to(store)) for a in (0.7, 0.3)]
    n = lambda v, norm: torch.tanh(norm[0] * v.double()) * norm[1].double() + norm[2].double()
    dev = [(a, w.cuda(), b.cuda()) for a, w, b in norms]
    tol = 2e-6 if dtype == "float32" else 1e-2
    out = rt.k.tanh_norm(x.cuda(), dev[0], torch.empty(rows, dim, dtype=rt.dtype, device="cuda"))
    want = n(x, norms[0])
    assert float((out.cpu().double() - want).abs().max()) <= tol * max(1.0, float(want.abs().max()))
    pick = torch.tensor([rows - 1, 0], dtype=torch.int32)
    out = rt.k.tanh_norm(x.cuda(), dev[0], torch.empty(2, dim, dtype=rt.dtype, device="cuda"), pick.cuda())
    assert float((out.cpu().double() - want[pick.long()]).abs().max()) <= tol * max(1.0, float(want.abs().max()))
    for following in (False, True):
        s = x.cuda().clone()
        values = torch.empty(rows, dim, dtype=rt.dtype, device="cuda")
        rt.k.tanh_norm_add(y.cuda(), dev[0], s, (dev[1], values) if following else None)
        total = x.double() + n(y, norms[0])
        assert float((s.cpu().double() - total).abs().max()) <= 2e-6 * max(1.0, float(total.abs().max()))     # 32-bit in both builds
        if following:
            want = n(total, norms[1])
            assert float((values.cpu().double() - want).abs().max()) <= tol * max(1.0, float(want.abs().max()))


@pytest.mark.parametrize("dtype", DTYPES)
def test_keys_read_from_another_layer_are_that_layers(folders, plain_logits, dtype):
    """A model whose later layer reads the keys of layer 1 under a mask of its own: the plain implementation with the
    mask of layer 1 there, or with its own queries' norm left out, gives other logits by far."""
    name = "A"
    (seq,) = sequences(name, [60], seed=21)
    cfg, W = P.load_plain(folders(name))
    eng = engine_for(folders(name), dtype, MODELS[name]["page"], pages_for(name, 60), max_seqs=1, max_seq_len=64)
    got, chose = run_schedule(eng, name, {"a": seq}, [[("a", 30)]] + [[("a", 1)] for _ in range(30)])
    assert_close(got["a"], plain_logits(name, seq, dtype, chose["a"]), dtype, "keys read from another layer")
    ref = P.forward_logits(cfg, W, seq).float()
    other = dict(cfg, layers=[dict(L) for L in cfg["layers"]])
    other["layers"][3] = dict(other["layers"][3], mixer=dict(other["layers"][3]["mixer"], mask={"size": 7, "keep_first": 3}))
    assert float((P.forward_logits(other, W, seq).float() - ref)[20:].abs().max()) > 20 * tolerance("float32", ref)
