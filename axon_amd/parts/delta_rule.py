"""The gated delta rule (the linear attention of Gated-DeltaNet-like models), with its state in the cache manager's
state slots.

From the input h one product gives [q | k | v | beta | decay | gate]: q and k of kv_heads x dim, v and the gate of
heads x vdim, the others a number a head; head a uses query and key head a // (heads / kv_heads).  q, k and v pass a
causal convolution of `conv` taps per channel (no bias), then silu; q and k become vectors of length 1 a head,
x / sqrt(sum(x^2) + 1e-6), q also times dim^(-1/2).  With beta = sigmoid(.) and
g = exp(-exp(A_log) softplus(. + dt_bias)), per head

    S <- g S,  u = beta (v - S^T k),  S <- S + k u^T,  o = S^T q          (S: dim x vdim, zero at first)

and the output is W_o (o / sqrt(mean(o^2) + eps) head by head, times a gain of vdim shared by the heads, times
act(gate)).  Two variations: `decay` = {"rank": r}, a decay a head and key channel, g = exp(-exp(A_log) softplus(W_a2 W_a1 h
+ dt_bias)) (dt_bias and W_a2's rows heads x dim, A_log a number a head; S <- diag(g) S); `gate` = {"rank": r}, the gate
W_g2 W_g1 h.  Their second products are 32-bit.  The product's rows, the convolutions' results, the step sizes, the state and the norm are 32-bit; a
request's state row holds S and the convolutions' last conv - 1 inputs, twice: the state behind position p in copy
p & 1, so that a decoding step reads one copy and writes the other and may be run again with the same result.  Long stretches of tokens run in chunks on the
32-bit matrix cores where the sizes allow (`step_chunks`): the same sums in another order.

Parameters: `hidden_size`, `heads`, `kv_heads`, `dim`, `vdim`, `conv`, `eps`, `decay`, `gate` (above; None: one product),
`gate_act` ("silu", the default, or "sigmoid"), `names` (the tensors' names under the
prefix: scope "mix.", q, k, v, b, a or a1 and a2, g or g1 and g2, A_log, dt_bias, norm, o; a convolution is the name + ".conv").
`forward(..., accumulate=False)` stores the 32-bit output instead of adding it.
"""
from __future__ import annotations

from typing import List, Optional, Tuple

import torch

from ..config.base import ConfigError
from ..kernels import MODE_ADD_F32, MODE_STORE_F32
from .base import CacheBinding, Mixer, StateSpec, TensorDecl, register_mixer
from .recurrent import step_spans


CHUNK = 64             # tokens of a chunk of the matrix-core form
LONG = 24              # a request's tokens of a step from which that form is used


def step_chunks(ctx) -> Optional[Tuple]:
    """The long stretches of a step in chunks, and the other requests: ((chunks int32 [n, 2] = (first token, tokens),
    spans5 int32 [m, 5] = (slot, first token, tokens, first chunk, chunks)), spans int32 [k, 3] = (slot, first token,
    tokens) of the rest) on the device, made once a step; None where no stretch is long."""
    if ctx.decode_only or all(s.q_len < LONG for s in ctx.spans):
        return None
    made = ctx.shared.get("delta_rule_chunks")
    if made is None:
        chunks, spans5, rest = [], [], []
        for s in ctx.spans:
            if s.q_len < LONG:
                rest.append([s.slot, s.q_start, s.q_len])
                continue
            spans5.append([s.slot, s.q_start, s.q_len, len(chunks), -(-s.q_len // CHUNK)])
            chunks += [[s.q_start + at, min(CHUNK, s.q_len - at)] for at in range(0, s.q_len, CHUNK)]
        put = lambda rows, width: torch.tensor(rows, dtype=torch.int32).view(-1, width).to(ctx.rt.device)
        made = ctx.shared["delta_rule_chunks"] = ((put(chunks, 2), put(spans5, 5)), put(rest, 3))
    return made


class GatedDeltaRule(Mixer):
    graph_safe = True
    stores_output = True

    def __init__(self, params, prefix=""):
        super().__init__(params, prefix)
        p = params
        self.hidden, self.heads, self.kv_heads = int(p["hidden_size"]), int(p["heads"]), int(p["kv_heads"])
        self.dim, self.vdim, self.taps, self.eps = int(p["dim"]), int(p["vdim"]), int(p["conv"]), float(p["eps"])
        if self.kv_heads < 1 or self.heads % self.kv_heads:
            raise ConfigError(f"{self.heads} heads are not a multiple of {self.kv_heads} query/key heads")
        if not 1 <= self.dim <= 256:
            raise ConfigError(f"the delta rule with keys of {self.dim} dims: the scan's kernel takes 1 to 256")
        if self.taps < 1:
            raise ConfigError(f"a convolution of {self.taps} taps")
        self.qk, self.inner = self.kv_heads * self.dim, self.heads * self.vdim
        self.channels = 2 * self.qk + self.inner                   # what the convolutions see: q, k, v
        rank = lambda key: int(p[key]["rank"]) if p.get(key) else 0
        self.decay_rank, self.gate_rank, self.gate_act = rank("decay"), rank("gate"), p.get("gate_act", "silu")
        if self.decay_rank < 0 or self.gate_rank < 0 or self.gate_act not in ("silu", "sigmoid"):
            raise ConfigError(f"the delta rule with ranks {self.decay_rank} and {self.gate_rank}, a gate through '{self.gate_act}'")
        # the product's rows: q, k, v, beta, the decay (or the first half of its low-rank product), the gate (likewise)
        self.first = ["q", "k", "v", "b", "a1" if self.decay_rank else "a", "g1" if self.gate_rank else "g"]
        self.beta_at, self.decay_at = self.channels, self.channels + self.heads
        self.gate_at = self.decay_at + (self.decay_rank or self.heads)
        self.rows_width = self.gate_at + (self.gate_rank or self.inner)
        self.tail_at = self.inner * self.dim                       # a copy of the state: S, then the kept inputs
        self.copy_elems = -(-(self.tail_at + (self.taps - 1) * self.channels) // 4) * 4
        names = p.get("names", {})
        base = prefix + names.get("scope", "mix.")
        self.n = {k: base + names.get(k, k) for k in ("q", "k", "v", "b", "a", "a1", "a2", "g", "g1", "g2", "A_log", "dt_bias", "norm", "o")}

    def tensors(self) -> List[TensorDecl]:
        n, W = self.n, self.hidden
        widths = {"q": self.qk, "k": self.qk, "v": self.inner, "b": self.heads, "a": self.heads, "a1": self.decay_rank, "g": self.inner,
                  "g1": self.gate_rank}
        decays = self.heads * self.dim if self.decay_rank else self.heads
        second = [TensorDecl(n["a2"], (decays, self.decay_rank))] if self.decay_rank else []
        second += [TensorDecl(n["g2"], (self.inner, self.gate_rank))] if self.gate_rank else []
        return ([TensorDecl(n[k], (widths[k], W)) for k in self.first] + second
                + [TensorDecl(n[k] + ".conv", (widths[k], self.taps)) for k in ("q", "k", "v")]
                + [TensorDecl(n["A_log"], (self.heads,), "bias"), TensorDecl(n["dt_bias"], (decays,), "bias"),
                   TensorDecl(n["norm"], (self.vdim,), "gain"), TensorDecl(n["o"], (W, self.inner))])

    def state_spec(self) -> StateSpec:
        return StateSpec(2 * self.copy_elems)

    def input_projections(self):
        widths = {"q": self.qk, "k": self.qk, "v": self.inner, "b": self.heads, "a": self.heads, "a1": self.decay_rank, "g": self.inner,
                  "g1": self.gate_rank}
        return [(self.n[k], widths[k], None) for k in self.first]

    def load(self, store, rt, own_input: bool = True) -> None:
        n = self.n
        if own_input:
            self.w_in = rt.k.prepare_weight(store.fused_matrix([n[k] for k in self.first]))
        self.w_decay = store.matrix(n["a2"]) if self.decay_rank else None
        self.w_gate = store.matrix(n["g2"]) if self.gate_rank else None
        self.conv_w = store.fused_matrix([n[k] + ".conv" for k in ("q", "k", "v")])
        self.a_log, self.dt_bias, self.gain = store.vector(n["A_log"]), store.vector(n["dt_bias"]), store.vector(n["norm"])
        self.w_o = rt.k.prepare_weight(store.matrix(n["o"]))
        store.forget(n["o"])

    def forward(self, ctx, binding: CacheBinding, h, out, accumulate: bool = True, rows=None) -> None:
        k, T, f32 = ctx.rt.k, h.shape[0], torch.float32
        state = ctx.cache.state(binding.state_index)
        if rows is None:
            rows = ctx.ws.take((T, self.rows_width), f32)
            k.gemm(h, self.w_in, rows, None, MODE_STORE_F32)
        u, terms = ctx.ws.take((T, self.channels), f32), ctx.ws.take((T, self.heads, 2), f32)
        k.delta_prepare(rows, self.conv_w, state, self.copy_elems, self.tail_at, ctx.positions, ctx.seq_rows, self.beta_at, self.decay_at,
                        None if self.decay_rank else self.a_log, None if self.decay_rank else self.dt_bias, u, terms, self.heads, self.kv_heads, self.dim, self.vdim, self.dim ** -0.5)
        decay, gate = None, rows[:, self.gate_at:self.rows_width]
        if self.decay_rank:
            decay = ctx.ws.take((T, self.heads * self.dim), f32)
        if self.gate_rank:
            gate = ctx.ws.take((T, self.inner), f32)
        if self.decay_rank or self.gate_rank:
            k.delta_low_rank(rows, decay=(self.decay_at, self.w_decay, self.dt_bias, self.a_log, decay) if self.decay_rank else None,
                             gate=(self.gate_at, self.w_gate, gate) if self.gate_rank else None)
        y = ctx.ws.take((T, self.inner), f32)
        long = step_chunks(ctx) if k.delta_chunked_ok(self.kv_heads, self.heads, self.dim, self.vdim) else None
        chunks, spans = long if long is not None else (None, step_spans(ctx))
        k.delta_scan(u, terms, state, self.copy_elems, self.tail_at, spans, ctx.positions, ctx.seq_rows, rows, y, self.heads,
                     self.kv_heads, self.dim, self.vdim, self.taps, chunks=chunks, decay=decay)
        gated = ctx.ws.take((T, self.inner), ctx.rt.dtype)
        k.head_norm_gate(y, gate, self.gain, self.eps, gated, self.heads, act=self.gate_act)
        k.gemm(gated, self.w_o, out, None, MODE_ADD_F32 if accumulate else MODE_STORE_F32)


register_mixer("gated_delta_rule", GatedDeltaRule)
