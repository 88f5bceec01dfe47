"""The Lilunex decoder, slowly and plainly: whole sequences, no cache, float64.

One function per mechanism, written from the design's equations and sharing nothing with the
engine.  A model is (cfg, W): config.json as a dict and the tensors by name as float64.

Notation: h is a [T, width] input, positions are 0 .. T - 1, sigma is the logistic function,
unit(x) = x / sqrt(mean(x^2) + eps), n_a(x) = tanh(alpha_a x) w_a + b_a (a norm without statistics).

    layer      : x <- x + n_1b(mixer(n_1(x)));  x <- x + n_2b(ff(n_2(x)))
    wkv        : each of r, k, v, g, w reads h + (h' - h) mu_s, h' the previous token's h (0 before the first);
                 w = exp(-exp(W_w2 tanh(W_w1 .) + w0)); per head o = (S + diag(u) k v^T)^T r, S <- diag(w) S + k v^T;
                 W_o ([unit(o) of every head] norm silu(W_g .))
    attention  : q, k unit over all their rows at once with a gain, the first `dims` places of a head turned in
                 pairs (i, i + dims / 2) by p base^(-2 i / dims) / factor; i sees j <= i with i - j < size or
                 j < keep_first; p_ij = exp(s_ij) / (exp(sink) + sum exp(s_ij')); W_o . + b_o; a layer may read
                 another layer's keys and values
    delta      : q, k, v through a causal convolution and silu, q and k of length 1 a head, q / sqrt(dim);
                 S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q; W_o (unit(o) norm silu(W_g h))
    dense      : W_down relu(W_up h)^2
    experts    : s = softmax(W_r h) over experts and identities; the `top` largest s + correction; weights s over
                 their sum; an identity gives h; plus sigma(w_sg . h) shared(h)
    output     : head n_final(x)
"""
import json
import math
import os

import torch


def load_plain(model_dir):
    from safetensors.torch import load_file
    with open(os.path.join(model_dir, "config.json")) as f:
        cfg = json.load(f)
    W = {k: v.double() for k, v in load_file(os.path.join(model_dir, "model.safetensors")).items()}
    return cfg, W


# --------------------------------------------------------------------------- small pieces
def unit(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def sigma(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigma(z)


def softplus(z):
    return torch.where(z > 30.0, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def tanh_norm(W, name, x):
    return torch.tanh(W[name + ".alpha"] * x) * W[name] + W[name + ".b"]


# --------------------------------------------------------------------------- time mixing
def shifted(h):
    """The previous token's row for every row; zeros for the first."""
    return torch.cat([torch.zeros_like(h[:1]), h[:-1]])


def wkv_recurrence(r, k, v, w, u):
    """r, k, w [T, H, d], v [T, H, d], u [H, d] -> o [T, H, d]."""
    T, H, d = r.shape
    S = torch.zeros(H, d, v.shape[2], dtype=torch.float64)
    out = torch.zeros_like(v)
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out[t] = ((S + u[:, :, None] * kv) * r[t][:, :, None]).sum(dim=1)
        S = w[t][:, :, None] * S + kv
    return out


def wkv_mixer(W, p, c, h, eps):
    T = h.shape[0]
    H, d = c["heads"], c["dim"]
    back = shifted(h)
    mix = {s: h + (back - h) * W[p + "mu." + s] for s in "rkvgw"}
    r, k, v = ((mix[s] @ W[p + s].T).view(T, H, d) for s in "rkv")
    gate = silu(mix["g"] @ W[p + "g"].T)
    z = torch.tanh(mix["w"] @ W[p + "w1"].T) @ W[p + "w2"].T + W[p + "w0"]
    w = torch.exp(-torch.exp(z)).view(T, H, d)
    o = unit(wkv_recurrence(r, k, v, w, W[p + "u"]), eps).reshape(T, H * d)
    return (o * W[p + "norm"] * gate) @ W[p + "o"].T


# --------------------------------------------------------------------------- attention
def rotate_halves(v, positions, rot):
    """v [T, heads, dim]: the first rot.dims places of every head turn, place i with place i + dims / 2."""
    dims, base = int(rot["dims"]), float(rot["base"])
    factor = float((rot.get("scaling") or {}).get("factor", 1.0))
    half = dims // 2
    out = v.clone()
    for i in range(half):
        a = positions.double() * (base ** (-2.0 * i / dims) / factor)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        x, y = v[..., i], v[..., i + half]
        out[..., i] = x * c - y * s
        out[..., i + half] = y * c + x * s
    return out


def seen(T, mask):
    """[T, T] of bool: whether position i sees position j."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    ok = j <= i
    if mask:
        ok = ok & ((i - j < int(mask["size"])) | (j < int(mask["keep_first"])))
    return ok


def sink_softmax(s, sink):
    """s [..., T] with -inf where nothing is seen; exp(sink) joins the denominator."""
    m = torch.maximum(s.max(dim=-1, keepdim=True).values, sink)
    e = torch.exp(s - m)
    return e / (e.sum(dim=-1, keepdim=True) + torch.exp(sink - m))


def heads_attention(q, k, v, scale, mask, sinks):
    T, H, _ = q.shape
    G = k.shape[1]
    ok = seen(T, mask)
    out = torch.zeros(T, H, v.shape[2], dtype=torch.float64)
    for a in range(H):
        g = a // (H // G)
        s = torch.where(ok, (q[:, a] @ k[:, g].T) * scale, torch.tensor(-math.inf, dtype=torch.float64))
        out[:, a] = sink_softmax(s, sinks[a]) @ v[:, g]
    return out


def keys_and_values(W, p, c, h, eps):
    T = h.shape[0]
    G = c["kv_heads"]
    k = unit(h @ W[p + "k"].T + W[p + "k.b"], eps) * W[p + "k.norm"]
    k = k.view(T, G, c["dim"])
    v = (h @ W[p + "v"].T + W[p + "v.b"]).view(T, G, c["vdim"])
    rot = c.get("rot")
    return (rotate_halves(k, torch.arange(T), rot) if rot else k), v


def attention_mixer(W, p, c, h, eps, shared=None):
    """`shared`: the keys and values of another layer, which this one reads."""
    T = h.shape[0]
    H, d = c["heads"], c["dim"]
    q = (unit(h @ W[p + "q"].T + W[p + "q.b"], eps) * W[p + "q.norm"]).view(T, H, d)
    if c.get("rot"):
        q = rotate_halves(q, torch.arange(T), c["rot"])
    k, v = shared if shared is not None else keys_and_values(W, p, c, h, eps)
    o = heads_attention(q, k, v, float(c["scale"]), c.get("mask"), W[p + "sink"])
    return o.reshape(T, H * c["vdim"]) @ W[p + "o"].T + W[p + "o.b"]


# --------------------------------------------------------------------------- the delta rule
def causal_conv(x, w):
    """x [T, C], w [C, taps] (the last column is the current token's), zeros before the start."""
    T, C = x.shape
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, C, dtype=x.dtype), x])
    out = torch.zeros_like(x)
    for j in range(taps):
        out = out + padded[j:j + T] * w[:, j]
    return out


def unit_length(x):
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + 1e-6)


def delta_recurrence(q, k, v, g, beta):
    """q, k [T, H, d], v [T, H, dv], g, beta [T, H] -> o [T, H, dv]."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=torch.float64)
    out = torch.zeros_like(v)
    for t in range(T):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(dim=1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(dim=1)
    return out


def delta_mixer(W, p, c, h, eps):
    T = h.shape[0]
    H, G, d, dv = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q, k, v = (silu(causal_conv(h @ W[p + s].T, W[p + s + ".conv"])) for s in "qkv")
    q = unit_length(q.view(T, G, d)) * d ** -0.5
    k = unit_length(k.view(T, G, d))
    of = torch.arange(H) // (H // G)
    beta = sigma(h @ W[p + "b"].T)
    g = torch.exp(-torch.exp(W[p + "A_log"]) * softplus(h @ W[p + "a"].T + W[p + "dt_bias"]))
    o = delta_recurrence(q[:, of], k[:, of], v.view(T, H, dv), g, beta)
    o = unit(o, eps) * W[p + "norm"] * silu(h @ W[p + "g"].T).view(T, H, dv)
    return o.reshape(T, H * dv) @ W[p + "o"].T


# --------------------------------------------------------------------------- feed-forward
def dense_ff(W, p, h):
    return torch.relu(h @ W[p + "up"].T) ** 2 @ W[p + "down"].T


def gated_unit(W, p, h):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def router_scores(W, p, h):
    return torch.softmax(h @ W[p + "router"].T, dim=-1)


def choose_experts(choice, top):
    """The `top` largest choice scores of every row, of equal ones the lower expert."""
    return [sorted(range(len(s)), key=lambda e: (-s[e], e))[:top] for s in choice.tolist()]


def experts_ff(W, p, c, h, forced=None, slack=0.0):
    """`forced`: per position the experts another implementation chose; they are taken if each of them
    would be among the chosen with `slack` added to its score (a close call), else the run fails."""
    scores = router_scores(W, p, h)
    choice = scores + W[p + "correction"]
    n, top = int(c["router"]["experts"]), int(c["router"]["top"])
    chosen = choose_experts(choice, top)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        mine = chosen[t]
        if forced is not None and sorted(forced[t]) != sorted(mine):
            floor = min(float(choice[t, e]) for e in mine)
            if any(float(choice[t, e]) + slack < floor for e in forced[t]):
                raise AssertionError(f"{p} position {t}: experts {forced[t]} are no close call of {mine}")
            mine = forced[t]
        total = sum(float(scores[t, e]) for e in mine) + 1e-20
        for e in mine:
            y = gated_unit(W, f"{p}e{e}.", h[t][None])[0] if e < n else h[t]
            out[t] += scores[t, e] / total * y
    if c.get("shared"):
        out = out + sigma(h @ W[p + "shared.sg"].T) * gated_unit(W, p + "shared.", h)
    return out


# --------------------------------------------------------------------------- the model
def residual_stream(cfg, W, tokens, after_every_layer=None, forced=None, slack=0.0):
    eps = float(cfg["norm"]["eps"])
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)] * float(cfg["embedding"]["scale"])
    kept = {}
    for i, L in enumerate(cfg["layers"]):
        p, c = f"l{i}.", L["mixer"]
        h = tanh_norm(W, p + "norm1", x)
        if L["type"] == "wkv":
            y = wkv_mixer(W, p + "mix.", c, h, eps)
        elif L["type"] == "attention":
            if c.get("kv_from") is None:
                kept[i] = keys_and_values(W, p + "mix.", c, h, eps)
            y = attention_mixer(W, p + "mix.", c, h, eps, kept[i if c.get("kv_from") is None else c["kv_from"]])
        elif L["type"] == "delta":
            y = delta_mixer(W, p + "mix.", c, h, eps)
        else:
            raise ValueError(L["type"])
        x = x + tanh_norm(W, p + "norm1b", y)
        mlp = L.get("mlp")
        if mlp is not None:
            h = tanh_norm(W, p + "norm2", x)
            y = dense_ff(W, p + "mlp.", h) if mlp["kind"] == "dense" else \
                experts_ff(W, p + "mlp.", mlp, h, None if forced is None else forced.get(i), slack)
            x = x + tanh_norm(W, p + "norm2b", y)
        if after_every_layer is not None:
            after_every_layer.append(x.clone())
    return x


def forward_logits(cfg, W, tokens, forced=None, slack=0.0):
    return tanh_norm(W, "final.norm", residual_stream(cfg, W, tokens, forced=forced, slack=slack)) @ W["head"].T


def greedy_generate(cfg, W, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(forward_logits(cfg, W, seq)[-1].argmax()))
    return seq[len(prompt):]
