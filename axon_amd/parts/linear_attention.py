"""Linear attention with a constant decay a head ("lightning attention"), with its state in the cache manager's state slots.

q = silu(W_q h), k = silu(W_k h) (heads x dim), v = silu(W_v h) (heads x vdim).  Per head

    S_t = decay_h S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t                    (S: dim x vdim, zero at first)

and the output is W_o (o / sqrt(mean(o^2) + eps) over all heads at once, times a gain of heads vdim, times
sigmoid(W_g h)).  The products' rows, the state and the norm are 32-bit; a request's state row holds S twice: the state
behind position p in copy p & 1, so that a decoding step reads one copy and writes the other and may be run again with the
same result.  Long stretches of tokens run in chunks on the 32-bit matrix cores where the sizes allow: the same sums in
another order.

Parameters: `hidden_size`, `heads`, `dim`, `vdim`, `decay` (a number a head), `eps`, `names` (the tensors' names under the
prefix: scope "mix.", q, k, v, g, o, norm).  `forward(..., accumulate=False)` stores the 32-bit output instead of adding it.
"""
from __future__ import annotations

from typing import List

import torch

from ..config.base import ConfigError
from ..kernels import MODE_ADD_F32, MODE_STORE_F32
from .base import CacheBinding, Mixer, StateSpec, TensorDecl, register_mixer
from .delta_rule import step_chunks
from .recurrent import step_spans


class LightningAttention(Mixer):
    graph_safe = True
    stores_output = True

    def __init__(self, params, prefix=""):
        super().__init__(params, prefix)
        p = params
        self.hidden, self.heads, self.dim, self.vdim = int(p["hidden_size"]), int(p["heads"]), int(p["dim"]), int(p["vdim"])
        self.eps = float(p["eps"])
        self.decays = [float(d) for d in p["decay"]]
        if len(self.decays) != self.heads:
            raise ConfigError(f"{len(self.decays)} decays for {self.heads} heads of linear attention")
        if not 1 <= self.dim <= 256:
            raise ConfigError(f"linear attention with keys of {self.dim} dims: the scan's kernel takes 1 to 256")
        self.qk, self.inner = self.heads * self.dim, self.heads * self.vdim
        self.gate_at = 2 * self.qk + self.inner                    # the product's rows: q, k, v, the gate
        self.copy_elems = -(-self.inner * self.dim // 4) * 4
        names = p.get("names", {})
        base = prefix + names.get("scope", "mix.")
        self.n = {k: base + names.get(k, k) for k in ("q", "k", "v", "g", "o", "norm")}

    def tensors(self) -> List[TensorDecl]:
        n, W = self.n, self.hidden
        widths = {"q": self.qk, "k": self.qk, "v": self.inner, "g": self.inner}
        return [TensorDecl(n[k], (rows, W)) for k, rows in widths.items()] + [TensorDecl(n["norm"], (self.inner,), "gain"),
                                                                              TensorDecl(n["o"], (W, self.inner))]

    def state_spec(self) -> StateSpec:
        return StateSpec(2 * self.copy_elems)

    def input_projections(self):
        widths = {"q": self.qk, "k": self.qk, "v": self.inner, "g": self.inner}
        return [(self.n[k], rows, None) for k, rows in widths.items()]

    def load(self, store, rt, own_input: bool = True) -> None:
        n = self.n
        if own_input:
            self.w_in = rt.k.prepare_weight(store.fused_matrix([n[k] for k in ("q", "k", "v", "g")]))
        self.gain = store.vector(n["norm"])
        self.decay = torch.tensor(self.decays, dtype=torch.float32, device=rt.device)
        self.w_o = rt.k.prepare_weight(store.matrix(n["o"]))
        store.forget(n["o"])

    def forward(self, ctx, binding: CacheBinding, h, out, accumulate: bool = True, rows=None) -> None:
        k, T, f32 = ctx.rt.k, h.shape[0], torch.float32
        state = ctx.cache.state(binding.state_index)
        if rows is None:
            rows = ctx.ws.take((T, self.gate_at + self.inner), f32)
            k.gemm(h, self.w_in, rows, None, MODE_STORE_F32)
        y = ctx.ws.take((T, self.inner), f32)
        chunks_ok = rows.data_ptr() % 16 == 0 and k.lightning_chunked_ok(self.heads, self.dim, self.vdim, rows.stride(0), 0, self.qk)
        long = step_chunks(ctx) if chunks_ok else None
        chunks, spans = long if long is not None else (None, step_spans(ctx))
        if chunks is not None:
            k.silu_rows(rows, self.gate_at)
        k.lightning_scan(rows, 0, self.qk, 2 * self.qk, chunks is None, self.decay, state, self.copy_elems, spans, ctx.positions,
                         ctx.seq_rows, y, self.heads, self.dim, self.vdim, chunks=chunks)
        gated = ctx.ws.take((T, self.inner), ctx.rt.dtype)
        k.head_norm_gate(y, rows[:, self.gate_at:self.gate_at + self.inner], self.gain, self.eps, gated, 1, act="sigmoid")
        k.gemm(gated, self.w_o, out, None, MODE_ADD_F32 if accumulate else MODE_STORE_F32)


register_mixer("lightning_attention", LightningAttention)
