"""Small Lilunex configurations and weights for the tests: sizes that differ between the models and between the
layers of a model (key size against value size, heads against key/value heads, keys against values of a state),
values of 1 (one head, one tap, one expert a token, a window of one position), every expert chosen, more identities
than experts, no identities, no shared expert, no feed-forward, fewer rotated places than a head holds or none, no
scaling, no mask, windows shorter than the kept positions, no kept positions, windows beyond every sequence, layers that
read an earlier layer's keys with a mask wider, narrower or of more kept positions than that layer's own, sizes that no
matrix-core product takes and sizes that the matrix-core attention takes, states of more rows than a lane holds at
once, and weights drawn so that the mechanisms matter: decays from a step to hundreds of steps, scores of the size of
the sinks, routers whose corrections change the choice."""
import json
import os

import torch


def wkv(heads, dim):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim}}


def att(heads, kv_heads, dim, vdim, mask=None, rot=None, kv_from=None, scale=None):
    """mask: (size, keep_first); rot: (dims, base, factor or None)."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale else dim ** -0.5}
    if mask is not None:
        m["mask"] = {"size": mask[0], "keep_first": mask[1]}
    if rot is not None:
        m["rot"] = {"base": rot[1], "dims": rot[0]}
        if rot[2] is not None:
            m["rot"]["scaling"] = {"factor": rot[2]}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m}


def delta(heads, kv_heads, dim, vdim, conv=4):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, identity, top, ff, shared=None):
    m = {"kind": "moe", "router": {"experts": experts, "identity": identity, "top": top}, "expert": {"ff": ff}}
    if shared is not None:
        m["shared"] = {"ff": shared}
    return m


def layer(mixer, mlp):
    return dict(mixer, mlp=mlp)


def config(width, vocab, layers, eps=1e-5, scale=1.0):
    return {"architecture": "Lilunex", "embedding": {"scale": scale}, "layers": layers, "norm": {"eps": eps}, "vocab": vocab,
            "width": width}


MODELS = {
    # nothing a multiple of 16, pages of 8: a window of seven positions beside three kept ones, read again under a wider
    # window with more kept ones; four of ten places rotated; a layer without a feed-forward
    "A": dict(cfg=config(42, 131, [
        layer(wkv(3, 5), dense(50)),
        layer(att(4, 2, 10, 6, mask=(7, 3), rot=(4, 100.0, 2.0)), moe(5, 2, 2, 24, shared=16)),
        layer(delta(3, 1, 7, 5, conv=2), None),
        layer(att(6, 2, 10, 6, mask=(12, 9), rot=(4, 100.0, 2.0), kv_from=1), dense(24)),
        layer(wkv(1, 9), moe(2, 3, 4, 10))], scale=1.5), page=8, rank={0: 3, 4: 1}, seed=3),
    # what the matrix cores take, pages of 64: windows that end inside a page, keys read again without a window's kept
    # positions; every expert chosen; a state of 64 rows
    "B": dict(cfg=config(128, 300, [
        layer(att(8, 2, 32, 48, mask=(70, 4), rot=(32, 10000.0, 4.0)), dense(192)),
        layer(delta(4, 2, 64, 32, conv=4), moe(4, 0, 4, 64, shared=96)),
        layer(wkv(4, 32), moe(6, 2, 3, 32, shared=32)),
        layer(att(16, 16, 64, 16, mask=(40, 66), rot=(16, 500.0, None)), dense(128)),
        layer(att(4, 2, 32, 48, mask=(130, 0), rot=(32, 10000.0, 4.0), kv_from=0), moe(4, 4, 1, 64)),
        layer(att(16, 16, 64, 16, mask=(9, 2), rot=(16, 500.0, None), kv_from=3), None)], eps=1e-6, scale=2.0),
        page=64, rank={2: 64}, seed=8),
    # states of more rows than sixteen lanes hold at eight each, one tap, heads as many as query/key heads, a window of
    # one position, kept positions beyond the window's size, one expert a token, pages of 16
    "C": dict(cfg=config(64, 257, [
        layer(delta(2, 2, 132, 24, conv=1), moe(6, 1, 1, 32, shared=8)),
        layer(wkv(2, 70), dense(40)),
        layer(att(2, 1, 24, 40, mask=(1, 20), rot=(24, 50.0, 8.0)), moe(3, 1, 2, 16, shared=24)),
        layer(att(5, 5, 8, 8, mask=(1000, 1)), dense(64))], eps=1e-4), page=16, rank={1: 16}, seed=5),
    # one head each, no rotation and no mask at all, an unmasked layer that reads windowed keys (which then have to stay)
    "D": dict(cfg=config(80, 140, [
        layer(att(1, 1, 24, 40, mask=(5, 0)), moe(8, 4, 3, 24)),
        layer(att(3, 1, 24, 40, kv_from=0), dense(56)),
        layer(delta(1, 1, 16, 40, conv=5), moe(2, 0, 2, 40, shared=40)),
        layer(wkv(1, 40), None),
        layer(att(6, 3, 16, 24, rot=(2, 7.0, 1.5)), dense(80))], eps=1e-6, scale=0.5), page=16, rank={3: 2}, seed=12),
    # recurrences alone: no pages at all
    "E": dict(cfg=config(64, 97, [
        layer(wkv(2, 32), dense(96)), layer(delta(4, 4, 32, 16, conv=3), dense(64)), layer(wkv(8, 8), moe(4, 1, 2, 32))], scale=1.25),
        page=16, rank={0: 16, 2: 5}, seed=21),
}


def draw_weights(cfg, seed, ranks=None):
    """name -> float32 tensor of values that bfloat16 holds exactly (both compute dtypes and the
    plain implementation then start from the same numbers)."""
    g = torch.Generator().manual_seed(seed)
    W = {}
    width = cfg["width"]

    def matrix(name, *shape, gain=1.0):
        W[name] = torch.randn(*shape, generator=g) * (gain / shape[-1] ** 0.5)

    def vector(name, *shape, mean=0.0, std=0.1):
        W[name] = torch.randn(*shape, generator=g) * std + mean

    def uniform(name, *shape, low, high):
        W[name] = torch.rand(shape, generator=g) * (high - low) + low

    def norm(name):
        vector(name, width, mean=1.0)
        vector(name + ".b", width)
        uniform(name + ".alpha", low=0.5, high=0.9)

    # small against what the layers add: the next token then depends on the earlier ones, not on the last alone
    W["embed"] = torch.randn(cfg["vocab"], width, generator=g) * 0.3
    matrix("head", cfg["vocab"], width)
    norm("final.norm")
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        norm(p + "norm1")
        norm(p + "norm1b")
        if L["type"] == "wkv":
            H, d = m["heads"], m["dim"]
            rank = (ranks or {}).get(i, 16)
            for s in "rkvgw":
                uniform(p + "mix.mu." + s, width, low=0.0, high=1.0)
            for s in "rkvg":
                matrix(p + "mix." + s, H * d, width, gain=1.5)
            matrix(p + "mix.w1", rank, width, gain=2.0)
            matrix(p + "mix.w2", H * d, rank, gain=0.7)
            # decays exp(-exp(w0)): from a step (w0 near 1.5) to hundreds of steps (near -6)
            uniform(p + "mix.w0", H * d, low=-6.0, high=1.5)
            vector(p + "mix.u", H, d, mean=0.5, std=0.5)
            vector(p + "mix.norm", H * d, mean=1.0)
            matrix(p + "mix.o", width, H * d)
        elif L["type"] == "attention":
            H, G = m["heads"], m["kv_heads"]
            sides = {"q": H * m["dim"]}
            if m.get("kv_from") is None:
                sides.update(k=G * m["dim"], v=G * m["vdim"])
            for s, rows in sides.items():
                matrix(p + "mix." + s, rows, width)
                vector(p + "mix." + s + ".b", rows, std=0.2)
                if s != "v":
                    vector(p + "mix." + s + ".norm", rows, mean=1.3, std=0.3)
            vector(p + "mix.sink", H, mean=1.0, std=1.0)
            matrix(p + "mix.o", width, H * m["vdim"], gain=1.5)
            vector(p + "mix.o.b", width, std=0.2)
        else:
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            for s, rows in (("q", G * d), ("k", G * d), ("v", H * dv)):
                matrix(p + "mix." + s, rows, width, gain=1.5)
                W[p + "mix." + s + ".conv"] = torch.randn(rows, m["conv"], generator=g) * 0.5 + 0.3
            matrix(p + "mix.b", H, width, gain=1.5)
            matrix(p + "mix.a", H, width)
            # decays from a step (A_log near 0.5) to hundreds of steps (near -5)
            uniform(p + "mix.A_log", H, low=-5.0, high=0.5)
            vector(p + "mix.dt_bias", H, mean=-0.5, std=0.5)
            matrix(p + "mix.g", H * dv, width, gain=1.5)
            vector(p + "mix.norm", dv, mean=1.0)
            matrix(p + "mix.o", width, H * dv)
        mlp = L.get("mlp")
        if mlp is None:
            continue
        norm(p + "norm2")
        norm(p + "norm2b")
        if mlp["kind"] == "dense":
            matrix(p + "mlp.up", mlp["ff"], width, gain=1.5)
            matrix(p + "mlp.down", width, mlp["ff"])
            continue
        E, I = mlp["router"]["experts"], mlp["router"]["identity"]
        matrix(p + "mlp.router", E + I, width, gain=2.0)
        vector(p + "mlp.correction", E + I, std=0.3)
        units = [(f"e{e}.", mlp["expert"]["ff"]) for e in range(E)]
        if mlp.get("shared"):
            units.append(("shared.", mlp["shared"]["ff"]))
            matrix(p + "mlp.shared.sg", 1, width, gain=2.0)
        for scope, ff in units:
            matrix(p + "mlp." + scope + "gate", ff, width, gain=2.0)
            matrix(p + "mlp." + scope + "up", ff, width, gain=2.0)
            matrix(p + "mlp." + scope + "down", width, ff)
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
