"""The Bafavik decoder, slowly and plainly: whole sequences, no cache, float64.

One function per mechanism, written from the design's equations and sharing nothing with the
engine.  A model is (cfg, W): config.json as a dict and the tensors by name as float64.

Notation: h is a [T, width] input, positions are 0 .. T - 1, sigma is the logistic function,
unit(x) = x / sqrt(mean(x^2) + eps), h'_t = h_(t-1) with h'_0 = 0.

    embedding  : x_t = embed[token_t] scale + bigram[(token_(t-1) mul_prev + token_t mul_cur) mod buckets];
                 bigram's last row for t = 0
    layer      : h = unit(x) (1 + norm1);  h <- h + (h' - h) shift;  x <- x + m ls1 mixer(h);
                 x <- x + m ls2 W_down relu(W_up (unit(x) (1 + norm2)))^2
    loop       : layers start .. stop - 1 run `times` times in a row
    parallel   : left_scale L + right_scale R
      L        : q, k, v with biases; halves of the first `dims` places turned; q, k <- unit per head; causal
                 softmax of q . k scale; W_o . + b_o
      R        : q, k, v <- silu(W h); S_t = decay_a S_(t-1) + k v^T; o = S_t^T q;  W_o (unit(heads side by side) norm sigma(W_g h))
    attention  : two maps a head over one set of values, in chunks of `size` positions; a = unit(a_1 - lam a_2) (1 - diff),
                 lam = exp(lq1 . lk1) - exp(lq2 . lk2) + diff;  W_o (a sigma(W_g h))
    parallel_2 : (unit(L) left.out + unit(R) right.out) / 2
      L        : q, k, v through a causal convolution; neighbours of the first `dims` places turned; causal softmax;
                 W_o (heads sigma(W_g h))
      R        : q, k, v through a causal convolution and silu, q and k of length 1 a head, q / sqrt(dim);
                 g = exp(-exp(A_log) softplus(W_a2 W_a1 h + dt_bias)) a head and key channel;
                 S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q;
                 W_o (unit(o) norm sigma(W_g2 W_g1 h))
    output     : head (unit(x) (1 + final.norm)) logit_scale
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


def around_zero_norm(W, name, x, eps):
    return unit(x, eps) * (1.0 + W[name])


def sigma(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigma(z)


def softplus(z):
    return torch.where(z > 30.0, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def shifted(h, share):
    """Every row moved towards the row before it (zeros before the first), a share a column."""
    before = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    return h + (before - h) * share


def causal_conv(x, w):
    """x [T, C], w [C, taps] (the last column is the current token's), zeros before the start."""
    T, C = x.shape
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, C, dtype=x.dtype), x])
    out = torch.zeros_like(x)
    for j in range(taps):
        out = out + padded[j:j + T] * w[:, j]
    return out


# --------------------------------------------------------------------------- embedding
def bigram_rows(tokens, bigram):
    """The row of the bigram table for every token of a sequence."""
    n, a, b = int(bigram["buckets"]), int(bigram["mul_prev"]), int(bigram["mul_cur"])
    return [n if t == 0 else (tokens[t - 1] * a + tokens[t] * b) % n for t in range(len(tokens))]


def embedding_rows(cfg, W, tokens):
    e = cfg["embedding"]
    tokens = [int(t) for t in tokens]
    x = W["embed"][torch.tensor(tokens)] * float(e["scale"])
    if e.get("bigram"):
        x = x + W["bigram"][torch.tensor(bigram_rows(tokens, e["bigram"]))]
    return x


# --------------------------------------------------------------------------- attention
def rotated(v, rot, neighbours):
    """v [T, heads, dim]: the first rot.dims places of every head turn by position, in pairs (2i, 2i + 1) or (i, i + dims / 2)."""
    if not rot:
        return v
    dims, base = int(rot["dims"]), float(rot["base"])
    p = torch.arange(v.shape[0], dtype=torch.float64)
    out = v.clone()
    for i in range(dims // 2):
        ia, ib = (2 * i, 2 * i + 1) if neighbours else (i, i + dims // 2)
        a = p * base ** (-2.0 * i / dims)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        x, y = v[..., ia], v[..., ib]
        out[..., ia] = x * c - y * s
        out[..., ib] = y * c + x * s
    return out


def seen(T, mask):
    """[T, T] of bool: whether position i sees position j."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    ok = j <= i
    if mask:
        ok = ok & (i // int(mask["size"]) == j // int(mask["size"]))
    return ok


def heads_attention(q, k, v, scale, mask):
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H, dv]: softmax over the keys a position sees."""
    T, H, _ = q.shape
    G = k.shape[1]
    ok = seen(T, mask)
    out = torch.zeros(T, H, v.shape[2], dtype=torch.float64)
    for a in range(H):
        g = a // (H // G)
        s = torch.where(ok, (q[:, a] @ k[:, g].T) * scale, torch.tensor(-math.inf, dtype=torch.float64))
        out[:, a] = torch.softmax(s, dim=-1) @ v[:, g]
    return out


def turned_normed_attention(W, p, c, h, eps):
    """The left side of "parallel": biases everywhere, rotation in halves, queries and keys of unit size behind it."""
    T, H, G, d = h.shape[0], c["heads"], c["kv_heads"], c["dim"]
    q, k, v = (h @ W[p + s].T + W[p + s + ".b"] for s in "qkv")
    q = unit(rotated(q.view(T, H, d), c.get("rot"), False), eps)
    k = unit(rotated(k.view(T, G, d), c.get("rot"), False), eps)
    o = heads_attention(q, k, v.view(T, G, c["vdim"]), float(c["scale"]), None)
    return o.reshape(T, H * c["vdim"]) @ W[p + "o"].T + W[p + "o.b"]


def convolved_attention(W, p, c, h):
    """The left side of "parallel_2": short convolutions, rotation in neighbours, a gate an element."""
    T, H, G, d = h.shape[0], c["heads"], c["kv_heads"], c["dim"]
    q, k, v = (causal_conv(h @ W[p + s].T, W[p + s + ".conv"]) for s in "qkv")
    q = rotated(q.view(T, H, d), c.get("rot"), True)
    k = rotated(k.view(T, G, d), c.get("rot"), True)
    o = heads_attention(q, k, v.view(T, G, c["vdim"]), float(c["scale"]), None)
    return (o.reshape(T, H * c["vdim"]) * sigma(h @ W[p + "g"].T)) @ W[p + "o"].T


def difference_factor(W, p, diff):
    dot = lambda a, b: torch.exp((W[p + a] * W[p + b]).sum())
    return dot("lq1", "lk1") - dot("lq2", "lk2") + diff


def differential_attention(W, p, c, h, eps):
    """The mixer "attention": two maps a head, chunks, no rotation, a gate an element."""
    T, H, G, d = h.shape[0], c["heads"], c["kv_heads"], c["dim"]
    q, k, v = (h @ W[p + s].T + W[p + s + ".b"] for s in "qkv")
    q, k, v = q.view(T, H, 2, d), k.view(T, G, 2, d), v.view(T, G, c["vdim"])
    diff = float(c["diff"])
    a1, a2 = (heads_attention(q[:, :, m], k[:, :, m], v, float(c["scale"]), c.get("mask")) for m in (0, 1))
    o = unit(a1 - difference_factor(W, p, diff) * a2, eps) * (1.0 - diff)
    return (o.reshape(T, H * c["vdim"]) * sigma(h @ W[p + "g"].T)) @ W[p + "o"].T


# --------------------------------------------------------------------------- recurrences
def lightning_recurrence(q, k, v, decay):
    """q, k [T, H, d], v [T, H, dv], decay [H] -> o [T, H, dv]; the read-out sees the token's own write."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=torch.float64)
    out = torch.zeros_like(v)
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(dim=1)
    return out


def lightning_mixer(W, p, c, h, eps):
    T, H, d, dv = h.shape[0], c["heads"], c["dim"], c["vdim"]
    q, k, v = (silu(h @ W[p + s].T) for s in "qkv")
    decay = torch.tensor([float(x) for x in c["decay"]], dtype=torch.float64)
    o = lightning_recurrence(q.view(T, H, d), k.view(T, H, d), v.view(T, H, dv), decay).reshape(T, H * dv)
    return (unit(o, eps) * W[p + "norm"] * sigma(h @ W[p + "g"].T)) @ W[p + "o"].T


def unit_length(x):
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + 1e-6)


def delta_recurrence(q, k, v, g, beta):
    """q, k, g [T, H, d], v [T, H, dv], beta [T, H] -> o [T, H, dv]; a decay for every row of the state."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=torch.float64)
    out = torch.zeros_like(v)
    for t in range(T):
        S = g[t][:, :, None] * S
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
    z = (h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "dt_bias"]
    g = torch.exp(-torch.exp(W[p + "A_log"])[:, None] * softplus(z).view(T, H, d))
    o = unit(delta_recurrence(q[:, of], k[:, of], v.view(T, H, dv), g, beta), eps) * W[p + "norm"]
    gate = sigma((h @ W[p + "g1"].T) @ W[p + "g2"].T)
    return (o.reshape(T, H * dv) * gate) @ W[p + "o"].T


# --------------------------------------------------------------------------- the model
def mixer(W, p, L, h, eps):
    c = L["mixer"]
    if L["type"] == "parallel":
        return (float(c["left_scale"]) * turned_normed_attention(W, p + "left.", c["left"], h, eps)
                + float(c["right_scale"]) * lightning_mixer(W, p + "right.", c["right"], h, eps))
    if L["type"] == "parallel_2":
        left, right = convolved_attention(W, p + "left.", c["left"], h), delta_mixer(W, p + "right.", c["right"], h, eps)
        return 0.5 * (unit(left, eps) * W[p + "left.out"] + unit(right, eps) * W[p + "right.out"])
    if L["type"] == "attention":
        return differential_attention(W, p, c, h, eps)
    raise ValueError(L["type"])


def squared_relu_ff(W, p, h):
    return torch.relu(h @ W[p + "up"].T) ** 2 @ W[p + "down"].T


def run_order(cfg):
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b = int(loop["start"]), int(loop["stop"])
    return list(range(a)) + list(range(a, b)) * int(loop["times"]) + list(range(b, n))


def residual_stream(cfg, W, tokens, after_every_run=None):
    eps, m = float(cfg["norm"]["eps"]), float(cfg.get("residual_mult", 1.0))
    x = embedding_rows(cfg, W, tokens)
    for i in run_order(cfg):
        p, L = f"l{i}.", cfg["layers"][i]
        h = shifted(around_zero_norm(W, p + "norm1", x, eps), W[p + "shift"])
        x = x + m * W[p + "ls1"] * mixer(W, p + "mix.", L, h, eps)
        if L.get("mlp") is not None:
            x = x + m * W[p + "ls2"] * squared_relu_ff(W, p + "mlp.", around_zero_norm(W, p + "norm2", x, eps))
        if after_every_run is not None:
            after_every_run.append(x.clone())
    return x


def forward_logits(cfg, W, tokens):
    x = residual_stream(cfg, W, tokens)
    h = around_zero_norm(W, "final.norm", x, float(cfg["norm"]["eps"]))
    return (h @ W["head"].T) * float(cfg.get("logit_scale", 1.0))


def greedy_generate(cfg, W, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(forward_logits(cfg, W, seq)[-1].argmax()))
    return seq[len(prompt):]
