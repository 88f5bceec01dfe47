"""Two mixers side by side on the same input: the result is the sum of their outputs, each normed or scaled.

Each side is a mixer of its own (a `PartSpec`), run on the same rows h.  `combine`:

* "normed": mult (rms(left(h)) g_l + rms(right(h)) g_r), an RMS norm over the model width with a plain gain and the
  layer's eps a side, times `mult` (a half: the mean of the two);
* "scaled": scales[0] left(h) + scales[1] right(h).

Where both sides take their projections of h ready made, one product makes them for both.  Norm, factors and the sum into the
residual stream are one 32-bit pass.  One side may keep pages (a `CacheSpec`); per-request
state either side may have (the run's binding holds the left side's arenas, then the right side's).

Parameters: `hidden_size`, `left`, `right` (the sides' PartSpecs; their tensors lie under
`<scope>left.` and `<scope>right.`), `combine` (default "normed"), `eps` and `mult` (default 0.5) for "normed", `scales` for
"scaled", `names` (scope "mix.", left_out "left.out", right_out "right.out": the gains of the two norms).
"""
from __future__ import annotations

from typing import List, Optional

import torch

from ..config.base import ConfigError, PartSpec
from ..kernels import MODE_STORE_F32
from .base import CacheBinding, CacheSpec, Mixer, OutputTerm, StateSpec, TensorDecl, build_part, register_mixer
from .masked_attention import load_projections


class PairedMixers(Mixer):

    def __init__(self, params, prefix=""):
        super().__init__(params, prefix)
        p = params
        self.hidden, self.eps, self.mult = int(p["hidden_size"]), float(p.get("eps", 0.0)), float(p.get("mult", 0.5))
        self.combine = p.get("combine", "normed")
        if self.combine not in ("normed", "scaled"):
            raise ConfigError(f"a pair of mixers is not combined '{self.combine}' (normed, scaled)")
        self.scales = [float(s) for s in p["scales"]] if self.combine == "scaled" else [1.0, 1.0]
        names = p.get("names", {})
        base = prefix + names.get("scope", "mix.")
        self.gain_names = [base + names.get("left_out", "left.out"), base + names.get("right_out", "right.out")]
        self.sides = [build_part("mixer", s if isinstance(s, PartSpec) else PartSpec(s["kind"], s["params"]), prefix)
                      for s in (p["left"], p["right"])]
        for side in self.sides:
            if not getattr(side, "stores_output", False):
                raise ConfigError(f"a side of a pair of mixers must be able to store its output ({type(side).__name__} cannot)")
        if sum(s.cache_spec() is not None for s in self.sides) > 1:
            raise ConfigError("a pair of mixers shares one binding: one side may keep pages")
        self.graph_safe = all(getattr(s, "graph_safe", False) for s in self.sides)
        self.gains = [None, None]
        projections = [s.input_projections() for s in self.sides]
        self.projections = None if any(p is None for p in projections) else projections
        self.w_in = self.b_in = None

    # what the engine asks a mixer is answered by the side that it concerns
    def _first(self, method: str, *args):
        for side in self.sides:
            got = getattr(side, method)(*args)
            if got is not None:
                return got
        return None

    def cache_spec(self) -> Optional[CacheSpec]:
        return self._first("cache_spec")

    def state_specs(self) -> List[StateSpec]:
        return [spec for side in self.sides for spec in side.state_specs()]

    def state_spec(self) -> Optional[StateSpec]:
        specs = self.state_specs()
        return specs[0] if specs else None

    def max_context(self) -> Optional[int]:
        limits = [m for m in (s.max_context() for s in self.sides) if m is not None]
        return min(limits) if limits else None

    def decode_shape(self, positions):
        return self._first("decode_shape", positions)

    def decode_input(self, positions):
        return self._first("decode_input", positions)

    def decode_input_capacity(self, max_seqs: int, max_seq_len: int) -> int:
        return max(s.decode_input_capacity(max_seqs, max_seq_len) for s in self.sides)

    def decode_scratch(self, max_seqs: int, max_seq_len: int):
        return self._first("decode_scratch", max_seqs, max_seq_len)

    def tensors(self) -> List[TensorDecl]:
        t = [d for s in self.sides for d in s.tensors()]
        return t + [TensorDecl(name, (self.hidden,), "gain") for name in self.gain_names] if self.combine == "normed" else t

    def load(self, store, rt) -> None:
        if self.projections is not None:
            self.w_in, self.b_in = load_projections([p for side in self.projections for p in side], store, rt)
        for s in self.sides:
            if self.projections is not None:
                s.load(store, rt, own_input=False)
            else:
                s.load(store, rt)
        if self.combine == "normed":
            self.gains = [store.vector(name) for name in self.gain_names]
        else:
            self.gains = [torch.full((self.hidden,), s, dtype=torch.float32, device=rt.device) for s in self.scales]

    def output_terms(self) -> List[OutputTerm]:
        if self.combine == "normed":
            return [OutputTerm(gain, self.mult, self.eps) for gain in self.gains]
        return [OutputTerm(None, s) for s in self.scales]

    def forward_apart(self, ctx, binding: CacheBinding, h, outs) -> None:
        at, parts = 0, [{}, {}]
        if self.projections is not None:
            left, right = (sum(rows for _, rows, _ in side) for side in self.projections)
            rows = ctx.ws.take((h.shape[0], left + right), torch.float32)
            ctx.rt.k.gemm(h, self.w_in, rows, self.b_in, MODE_STORE_F32)
            parts = [{"rows": rows[:, :left]}, {"rows": rows[:, left:]}]
        for side, out, ready in zip(self.sides, outs, parts):
            n = len(side.state_specs())
            side.forward(ctx, binding.with_states(at, n), h, out, accumulate=False, **ready)
            at += n

    def forward(self, ctx, binding: CacheBinding, h, residual) -> None:
        k = ctx.rt.k
        outs = [ctx.ws.take(tuple(residual.shape), torch.float32) for _ in self.sides]
        self.forward_apart(ctx, binding, h, outs)
        if self.combine == "scaled":
            k.scaled_sum([(y, gain, None) for y, gain in zip(outs, self.gains)], residual)
            return
        for y, gain in zip(outs, self.gains):
            k.norm_add(y, gain, self.eps, self.mult, residual)


register_mixer("paired_mixers", PairedMixers)
