"""Small Bafavik configurations and weights for the tests: sizes that differ between the models and between the layers of a
model (key size against value size, heads against key/value heads, taps, ranks), values of 1 (one head, one tap, one bucket of
token pairs, rank 1, a loop that runs once, chunks of one position), no table of token pairs, no loop, no feed-forward, fewer
rotated places than a head holds or none, no mask, chunks beyond every sequence, factors of every size, sizes that no
matrix-core product takes and sizes that the matrix-core kernels take, states of more rows than a lane holds at once, and weights
drawn so that the mechanisms matter: decays from a step to hundreds of steps, token shifts over all of [0, 1]."""
import json
import os

import torch


def heads(h, kv_heads, dim, vdim, scale=None, **more):
    return {"heads": h, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale else dim ** -0.5, **more}


def rot(dims, base):
    return {"rot": {"dims": dims, "base": base}} if dims else {}


def diff_att(h, kv_heads, dim, vdim, chunk=None, diff=0.3, scale=None):
    return {"type": "attention", "mixer": heads(h, kv_heads, dim, vdim, scale, diff=diff, **({"mask": {"size": chunk}} if chunk else {}))}


def parallel(left, decay, dim, vdim, scales=(0.8, 0.9)):
    return {"type": "parallel", "mixer": {"left": left, "right": {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)},
                                          "left_scale": scales[0], "right_scale": scales[1]}}


def parallel_2(left, conv, delta_heads, delta_kv, dim, vdim, delta_conv):
    return {"type": "parallel_2", "mixer": {"left": dict(left, conv=conv), "right": {
        "heads": delta_heads, "kv_heads": delta_kv, "dim": dim, "vdim": vdim, "conv": delta_conv}}}


def layer(mixer, ff):
    return dict(mixer, mlp=None if ff is None else {"kind": "dense", "ff": ff})


def config(width, vocab, layers, eps=1e-5, scale=1.0, bigram=None, mult=0.7, logit_scale=1.5, loop=None):
    """bigram: (buckets, mul_prev, mul_cur); loop: (start, stop, times)."""
    c = {"architecture": "Bafavik", "embedding": {"scale": scale}, "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width,
         "residual_mult": mult, "logit_scale": logit_scale}
    if bigram is not None:
        c["embedding"]["bigram"] = dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))
    if loop is not None:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


MODELS = {
    # nothing a multiple of 16, pages of 8, a loop over a mixed stretch, a layer without a feed-forward
    "A": dict(cfg=config(42, 131, [
        layer(diff_att(4, 2, 10, 6, chunk=7), 50),
        layer(parallel(heads(3, 1, 9, 7, **rot(4, 100.0)), [0.5, 0.97], 5, 11), None),
        layer(parallel_2(heads(4, 2, 6, 10, **rot(6, 50.0)), 3, 3, 1, 7, 5, 2), 24)], scale=1.5, bigram=(13, 5, 3), loop=(1, 3, 2)),
        page=8, rank={"l2.mix.right.a1": 3, "l2.mix.right.g1": 5}, seed=3),
    # what the matrix cores take, pages of 64: chunks that end inside a page, values larger and smaller than keys, a loop that
    # starts with the first layer
    "B": dict(cfg=config(128, 300, [
        layer(parallel_2(heads(8, 2, 32, 64, **rot(32, 10000.0)), 4, 4, 2, 64, 32, 4), 192),
        layer(parallel(heads(4, 4, 64, 48, **rot(16, 500.0)), [0.4, 0.9, 0.99, 1.0], 32, 16, (1.2, 0.6)), 128),
        layer(diff_att(8, 2, 16, 32, chunk=70, diff=0.1), 64)], eps=1e-6, scale=2.0, bigram=(97, 31, 11), loop=(0, 2, 2), mult=0.4),
        page=64, rank={"l0.mix.right.a1": 64, "l0.mix.right.g1": 16}, seed=8),
    # states of more rows than sixteen lanes hold at eight each, one tap, heads as many as query/key heads, one position a
    # chunk, no token pairs, no loop, pages of 16
    "C": dict(cfg=config(64, 257, [
        layer(parallel_2(heads(2, 1, 24, 40), 1, 2, 2, 132, 24, 1), 32),
        layer(parallel(heads(5, 5, 8, 8), [0.8], 140, 24, (0.5, 1.5)), 40),
        layer(diff_att(2, 1, 24, 40, chunk=1, diff=0.6), None),
        layer(diff_att(3, 3, 8, 24), 64)], eps=1e-4, mult=1.0, logit_scale=1.0), page=16,
        rank={"l0.mix.right.a1": 1, "l0.mix.right.g1": 70}, seed=5),
    # one head each, one bucket, a loop that runs once, five taps
    "D": dict(cfg=config(80, 140, [
        layer(parallel(heads(1, 1, 24, 40, **rot(2, 7.0)), [0.3, 0.999, 0.7], 16, 8), 24),
        layer(diff_att(1, 1, 16, 24, chunk=500), 56),
        layer(parallel_2(heads(6, 3, 16, 24, **rot(4, 20.0)), 5, 1, 1, 16, 40, 5), None)], scale=0.5, bigram=(1, 2, 3), loop=(2, 3, 1), mult=0.9),
        page=16, rank={"l2.mix.right.a1": 2, "l2.mix.right.g1": 2}, seed=12),
    # pairs alone, state keys of 96 and 128 rows in chunks, one model-wide loop
    "E": dict(cfg=config(64, 97, [
        layer(parallel(heads(2, 2, 32, 32, **rot(32, 10.0)), [0.95, 0.6], 128, 80), 96),
        layer(parallel_2(heads(4, 4, 32, 16, **rot(8, 300.0)), 2, 6, 3, 96, 48, 3), 64)], scale=1.25, bigram=(53, 7, 1), loop=(0, 2, 2)),
        page=64, rank={"l1.mix.right.a1": 16, "l1.mix.right.g1": 5}, seed=21),
}


def draw_weights(cfg, seed, ranks=None):
    """name -> float32 tensor of values that bfloat16 holds exactly (both compute dtypes and the plain implementation then
    start from the same numbers).  ranks: of the low-rank products by tensor name (16 where not named)."""
    g = torch.Generator().manual_seed(seed)
    W, ranks = {}, ranks or {}
    width = cfg["width"]

    def matrix(name, *shape, gain=1.0):
        W[name] = torch.randn(*shape, generator=g) * (gain / shape[-1] ** 0.5)

    def vector(name, *shape, mean=0.0, std=0.1):
        W[name] = torch.randn(*shape, generator=g) * std + mean

    def uniform(name, *shape, low, high):
        W[name] = torch.rand(shape, generator=g) * (high - low) + low

    def attention(p, m, maps=1, bias=(), gate=False, conv=0):
        H, G = m["heads"], m["kv_heads"]
        rows = {"q": H * maps * m["dim"], "k": G * maps * m["dim"], "v": G * m["vdim"]}
        for s, n in rows.items():
            matrix(p + s, n, width, gain=1.5)
            if s in bias:
                vector(p + s + ".b", n, std=0.3)
            if conv:
                W[p + s + ".conv"] = torch.randn(n, conv, generator=g) * 0.4 + (0.5 if conv > 1 else 0.8)
        if gate:
            matrix(p + "g", H * m["vdim"], width, gain=1.5)
        matrix(p + "o", width, H * m["vdim"], gain=1.5)
        if "o" in bias:
            vector(p + "o.b", width, std=0.2)

    W["embed"] = torch.randn(cfg["vocab"], width, generator=g) * 0.3
    if cfg["embedding"].get("bigram"):
        W["bigram"] = torch.randn(cfg["embedding"]["bigram"]["buckets"] + 1, width, generator=g) * 0.3
    matrix("head", cfg["vocab"], width)
    vector("final.norm", width, std=0.2)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        vector(p + "norm1", width, std=0.2)
        vector(p + "ls1", width, mean=0.8, std=0.3)
        uniform(p + "shift", width, low=0.0, high=1.0)
        if L["type"] == "attention":
            attention(p + "mix.", m, maps=2, bias="qkv", gate=True)
            for s in ("lq1", "lk1", "lq2", "lk2"):
                vector(p + "mix." + s, m["dim"], std=0.2)
        elif L["type"] == "parallel":
            attention(p + "mix.left.", m["left"], bias="qkvo")
            r, q = m["right"], p + "mix.right."
            for s, n in (("q", r["heads"] * r["dim"]), ("k", r["heads"] * r["dim"]), ("v", r["heads"] * r["vdim"]), ("g", r["heads"] * r["vdim"])):
                matrix(q + s, n, width, gain=1.5)
            matrix(q + "o", width, r["heads"] * r["vdim"], gain=1.5)
            vector(q + "norm", r["heads"] * r["vdim"], mean=1.0)
        else:
            attention(p + "mix.left.", m["left"], gate=True, conv=m["left"]["conv"])
            r, q = m["right"], p + "mix.right."
            H, G, d, dv = r["heads"], r["kv_heads"], r["dim"], r["vdim"]
            for s, rows in (("q", G * d), ("k", G * d), ("v", H * dv)):
                matrix(q + s, rows, width, gain=1.5)
                W[q + s + ".conv"] = torch.randn(rows, r["conv"], generator=g) * 0.5 + 0.3
            matrix(q + "b", H, width, gain=1.5)
            for first, second, rows in (("a1", "a2", H * d), ("g1", "g2", H * dv)):
                rank = ranks.get(q + first, 16)
                matrix(q + first, rank, width, gain=1.5)
                matrix(q + second, rows, rank, gain=1.5)
            # decays from a step (A_log near 0.5) to hundreds of steps (near -5)
            uniform(q + "A_log", H, low=-5.0, high=0.5)
            vector(q + "dt_bias", H * d, mean=-0.5, std=0.5)
            vector(q + "norm", dv, mean=1.0)
            matrix(q + "o", width, H * dv)
            for side in ("left", "right"):
                vector(p + f"mix.{side}.out", width, mean=1.0, std=0.2)
        if L.get("mlp") is not None:
            vector(p + "norm2", width, std=0.2)
            vector(p + "ls2", width, mean=0.8, std=0.3)
            matrix(p + "mlp.up", L["mlp"]["ff"], width, gain=1.5)
            matrix(p + "mlp.down", width, L["mlp"]["ff"])
    return {k: v.to(torch.bfloat16).float() for k, v in W.items()}


def write_model(path, cfg, W):
    from axon_amd.weights.safetensors_io import write_safetensors
    os.makedirs(path, exist_ok=True)
    write_safetensors(os.path.join(path, "model.safetensors"), [(k, v.to(torch.bfloat16)) for k, v in W.items()], {"format": "pt"})
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f, indent=1)
    return path


def make(path, name):
    m = MODELS[name]
    return write_model(path, m["cfg"], draw_weights(m["cfg"], m["seed"], m["rank"]))
