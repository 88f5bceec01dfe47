"""Time mixing with a state matrix a head (the time-mix block of RWKV-6-like models), with its state in the cache
manager's state slots.

Each of five uses of the input h (receptance r, key k, value v, gate g, decay w) reads a mix of a token's row and
the one before it, h + (h' - h) mu_s (h' = 0 before the first token).  r, k, v (heads x dim) and the gate are
products of their mixes; the decay is w = exp(-exp(w0 + W_w2 tanh(W_w1 mix_w))) per head and key channel.  Per head

    o_t = (S_(t-1) + diag(u) k_t v_t^T)^T r_t,   S_t = diag(w_t) S_(t-1) + k_t v_t^T     (S: dim x dim, zero at first)

and the output is W_o (o / sqrt(mean(o^2) + eps) head by head, times a gain of heads dim, times silu(gate)).  The
products' rows, the decay (with its low-rank product), the state and the norm are 32-bit; a request's state row
holds S and the last row of h, twice: the state behind position p in copy p & 1, so that a decoding step reads one
copy and writes the other and may be run again with the same result.  Where the walk of one chain a request would
leave most of the chip idle, a long stretch of tokens runs in segments side by side (`step_segments`): the same
sums in another order.

Parameters: `hidden_size`, `heads`, `dim`, `rank` (of the decay's low-rank product), `eps`, `names` (the tensors'
names under the prefix: scope "mix.", mu "mu.", r, k, v, g, w1, w2, w0, u, norm, o).  `forward(..., accumulate=False)`
stores the 32-bit output instead of adding it.
"""
from __future__ import annotations

from typing import List

import torch

from ..config.base import ConfigError
from ..kernels import MODE_ADD_F32, MODE_STORE_F32
from .base import CacheBinding, Mixer, StateSpec, TensorDecl, register_mixer
from .recurrent import step_spans
from .state_space import step_segments

USES = ("r", "k", "v", "g", "w")       # what reads a mix of its own, in the order of the shifted rows
VALUES_A_BLOCK = 16                    # value dims of a head a block of the walk takes


class TimeMix(Mixer):
    graph_safe = True
    stores_output = True

    def __init__(self, params, prefix=""):
        super().__init__(params, prefix)
        p = params
        self.hidden, self.heads, self.dim = int(p["hidden_size"]), int(p["heads"]), int(p["dim"])
        self.rank, self.eps = int(p["rank"]), float(p["eps"])
        if not 1 <= self.dim <= 256:
            raise ConfigError(f"time mixing with heads of {self.dim} dims: the scan's kernel takes 1 to 256")
        self.inner = self.heads * self.dim
        self.tail_at = self.inner * self.dim                       # a copy of the state: S, then the last row of h
        self.copy_elems = -(-(self.tail_at + self.hidden) // 4) * 4
        names = p.get("names", {})
        base = prefix + names.get("scope", "mix.")
        self.n = {k: base + names.get(k, k) for k in ("r", "k", "v", "g", "w1", "w2", "w0", "u", "norm", "o")}
        self.mu_names = [base + names.get("mu", "mu.") + s for s in USES]

    def tensors(self) -> List[TensorDecl]:
        n, W, C = self.n, self.hidden, self.inner
        return ([TensorDecl(name, (W,), "bias") for name in self.mu_names]
                + [TensorDecl(n[k], (C, W)) for k in ("r", "k", "v", "g")]
                + [TensorDecl(n["w1"], (self.rank, W)), TensorDecl(n["w2"], (C, self.rank)), TensorDecl(n["w0"], (C,), "bias"),
                   TensorDecl(n["u"], (self.heads, self.dim), "bias"), TensorDecl(n["norm"], (C,), "gain"), TensorDecl(n["o"], (W, C))])

    def state_spec(self) -> StateSpec:
        return StateSpec(2 * self.copy_elems)

    def load(self, store, rt) -> None:
        n = self.n
        self.mu = torch.stack([store.vector(name).float() for name in self.mu_names]).contiguous()
        self.w = {}
        for k in ("r", "k", "v", "g", "w1", "o"):
            self.w[k] = rt.k.prepare_weight(store.matrix(n[k]))
            store.forget(n[k])
        self.w2, self.w0 = store.matrix(n["w2"]), store.vector(n["w0"])
        self.u = store.vector(n["u"]).float().contiguous()
        self.gain = store.vector(n["norm"])

    def forward(self, ctx, binding: CacheBinding, h, out, accumulate: bool = True) -> None:
        k, T, C, f32 = ctx.rt.k, h.shape[0], self.inner, torch.float32
        state = ctx.cache.state(binding.state_index)
        mixed = ctx.ws.take((len(USES), T, self.hidden), ctx.rt.dtype)
        k.token_shift(h, self.mu, state, self.copy_elems, self.tail_at, ctx.positions, ctx.seq_rows, mixed)
        rows = ctx.ws.take((T, 4 * C), f32)
        for i, use in enumerate(("r", "k", "v", "g")):
            k.gemm(mixed[i], self.w[use], rows[:, i * C:(i + 1) * C], None, MODE_STORE_F32)
        low, decay = ctx.ws.take((T, self.rank), f32), ctx.ws.take((T, C), f32)
        k.gemm(mixed[4], self.w["w1"], low, None, MODE_STORE_F32)
        k.time_mix_decay(low, self.w2, self.w0, decay)
        y = ctx.ws.take((T, C), f32)
        k.wkv_scan(rows, 0, C, 2 * C, decay, self.u, state, self.copy_elems, self.tail_at, step_spans(ctx), ctx.positions, ctx.seq_rows,
                   h, y, self.heads, self.dim, self.dim, segments=step_segments(ctx, self.heads * -(-self.dim // VALUES_A_BLOCK)))
        gated = ctx.ws.take((T, C), ctx.rt.dtype)
        k.head_norm_gate(y, rows[:, 3 * C:], self.gain, self.eps, gated, self.heads)
        k.gemm(gated, self.w["o"], out, None, MODE_ADD_F32 if accumulate else MODE_STORE_F32)


register_mixer("time_mix", TimeMix)
