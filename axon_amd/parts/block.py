"""The arrangement of a layer's parts around the residual stream.

"prenorm": x += mixer(norm1(x)); x += feed_forward(norm2(x)), the order of
src/model.rs:2980-3055.  The residual stream `x` is float32 and is updated in place: the
mixer and the feed-forward add their output to it in the epilogue of their last product.
"""
from __future__ import annotations

from typing import List

import torch

from ..config.base import ConfigError
from .base import ROUNDED_STREAM, Block, CacheBinding, Mixer, Norm, OutputTerm, StateSpec, TensorDecl, register_block

# A norm behind a product whose kernel holds the finished rows anyway can be written by that
# kernel, and a norm before a product of few rows can be worked out inside that product (the same
# bits as the norm's own pass, both): the block asks its parts, step by step.


class PreNormBlock(Block):
    graph_safe = True
    norm1_name = "input_layernorm.weight"
    norm2_name = "post_attention_layernorm.weight"

    def __init__(self, norm_factory, mixer, feed_forward, prefix):
        super().__init__(norm_factory, mixer, feed_forward, prefix)
        self.norm1 = norm_factory(self.norm1_name)
        self.norm2 = norm_factory(self.norm2_name)

    def tensors(self) -> List[TensorDecl]:
        return self.norm1.tensors() + self.mixer.tensors() + self.norm2.tensors() + self.feed_forward.tensors()

    def load(self, store, rt) -> None:
        for part in (self.norm1, self.mixer, self.norm2, self.feed_forward):
            part.load(store, rt)

    def first_norm(self):
        return self.norm1

    def last_part(self):
        return self.feed_forward

    def forward(self, ctx, binding: CacheBinding, x, normed=None, following=None) -> None:
        h = normed
        if h is None:
            h = self.preceding_of(ctx, self.norm1, self.mixer, x)
        if h is None:
            h = self.norm1.forward(ctx, x)
        second = self.following_of(ctx, self.mixer, self.norm2, x.shape[0])
        if second is not None:
            self.mixer.forward(ctx, binding, h, x, second)
            h = second.values
        else:
            self.mixer.forward(ctx, binding, h, x)
            h = self.preceding_of(ctx, self.norm2, self.feed_forward, x)
            if h is None:
                h = self.norm2.forward(ctx, x)
        if following is not None:
            self.feed_forward.forward(ctx, h, x, following)
        else:
            self.feed_forward.forward(ctx, h, x)


class ShortNamedPreNormBlock(PreNormBlock):
    """The same arrangement for checkpoints that call the norms `norm1` and `norm2`; a layer may have no
    feed-forward (it then has no second norm either)."""
    norm1_name = "norm1"
    norm2_name = "norm2"

    def __init__(self, norm_factory, mixer, feed_forward, prefix):
        Block.__init__(self, norm_factory, mixer, feed_forward, prefix)
        self.norm1 = norm_factory(self.norm1_name)
        self.norm2 = norm_factory(self.norm2_name) if feed_forward is not None else None

    def parts(self):
        return [p for p in (self.norm1, self.mixer, self.norm2, self.feed_forward) if p is not None]

    def tensors(self) -> List[TensorDecl]:
        return [d for p in self.parts() for d in p.tensors()]

    def load(self, store, rt) -> None:
        for part in self.parts():
            part.load(store, rt)

    def last_part(self):
        return self.feed_forward if self.feed_forward is not None else self.mixer

    def forward(self, ctx, binding: CacheBinding, x, normed=None, following=None) -> None:
        if self.feed_forward is not None:
            return super().forward(ctx, binding, x, normed, following)
        h = normed
        if h is None:
            h = self.preceding_of(ctx, self.norm1, self.mixer, x)
        if h is None:
            h = self.norm1.forward(ctx, x)
        if following is not None:
            self.mixer.forward(ctx, binding, h, x, following)
        else:
            self.mixer.forward(ctx, binding, h, x)


class SublayerNormBlock(Block):
    """x += mult * norm1(mixer(x)); x += mult * norm2(feed_forward(x)): the norms sit on the sublayers'
    outputs, the sublayers read the residual stream itself (rounded to the compute dtype for their
    products), and a layer may have no feed-forward.  The norm, the scaling and the sum are one
    32-bit pass over the sublayer's 32-bit output, which also leaves the new rows rounded for the
    next sublayer.  The norms are RMS norms (they hand over a gain and an eps).  `residual_mult`
    comes with the norm's parameters."""
    graph_safe = True
    norm1_name = "norm1"
    norm2_name = "norm2"

    def __init__(self, norm_factory, mixer, feed_forward, prefix):
        super().__init__(norm_factory, mixer, feed_forward, prefix)
        self.norm1 = norm_factory(self.norm1_name)
        self.norm2 = norm_factory(self.norm2_name) if feed_forward is not None else None
        for norm in (self.norm1, self.norm2):
            if norm is not None and not (hasattr(norm, "gain") and hasattr(norm, "eps")):
                raise ConfigError("a norm on a sublayer's output is an RMS norm (a gain and an eps)")
        self.mult = float(self.norm1.params.get("residual_mult", 1.0))

    def parts(self):
        return [p for p in (self.norm1, self.mixer, self.norm2, self.feed_forward) if p is not None]

    def tensors(self) -> List[TensorDecl]:
        return [d for p in self.parts() for d in p.tensors()]

    def load(self, store, rt) -> None:
        for part in self.parts():
            part.load(store, rt)

    @staticmethod
    def _run(part, ctx, y, *args) -> None:
        """y = part(...): stored by the part's last product where it can, else added into zeros."""
        if getattr(part, "stores_output", False):
            part.forward(ctx, *args, y, accumulate=False)
        else:
            ctx.rt.k.fill_f32(y.view(-1), 0.0)
            part.forward(ctx, *args, y)

    def forward(self, ctx, binding: CacheBinding, x, normed=None, following=None) -> None:
        k, rt = ctx.rt.k, ctx.rt
        exact = rt.dtype == torch.float32            # the 32-bit path: the sublayers read x as it is
        h = x if exact else k.round_rows(x, ctx.ws.take(tuple(x.shape), rt.dtype))
        y = ctx.ws.take(tuple(x.shape), torch.float32)
        self._run(self.mixer, ctx, y, binding, h)
        if self.feed_forward is None:
            k.norm_add(y, self.norm1.gain, self.norm1.eps, self.mult, x)
            return
        h = x if exact else ctx.ws.take(tuple(x.shape), rt.dtype)
        k.norm_add(y, self.norm1.gain, self.norm1.eps, self.mult, x, None if exact else h)
        self._run(self.feed_forward, ctx, y, h)
        k.norm_add(y, self.norm2.gain, self.norm2.eps, self.mult, x)


class PostNormBlock(Block):
    """x <- norm1(alpha x + mixer(x)); x <- norm2(alpha x + feed_forward(x)): the norms sit behind the
    sums, the sublayers read the stream itself (rounded to the compute dtype for their products), and
    a layer may have no feed-forward (it then has no second norm).  The scaling, the sum and the norm
    are one 32-bit pass over the sublayer's 32-bit output, which also leaves the new rows rounded for
    the next sublayer, the next block's too.  The norms are RMS or layer norms (a gain, an eps and a
    `kind`); `stream_alpha` comes with the norm's parameters."""
    graph_safe = True
    norm1_name = "norm1"
    norm2_name = "norm2"

    def __init__(self, norm_factory, mixer, feed_forward, prefix):
        super().__init__(norm_factory, mixer, feed_forward, prefix)
        self.norm1 = norm_factory(self.norm1_name)
        self.norm2 = norm_factory(self.norm2_name) if feed_forward is not None else None
        for norm in (self.norm1, self.norm2):
            if norm is not None and not all(hasattr(norm, a) for a in ("gain", "eps", "kind")):
                raise ConfigError("a norm behind a sum is an RMS norm or a layer norm (a gain, an eps and a kind)")
        self.alpha = float(self.norm1.params.get("stream_alpha", 1.0))

    def parts(self):
        return [p for p in (self.norm1, self.mixer, self.norm2, self.feed_forward) if p is not None]

    def tensors(self) -> List[TensorDecl]:
        return [d for p in self.parts() for d in p.tensors()]

    def load(self, store, rt) -> None:
        for part in self.parts():
            part.load(store, rt)

    _run = staticmethod(SublayerNormBlock._run)

    def forward(self, ctx, binding: CacheBinding, x, normed=None, following=None) -> None:
        k, rt = ctx.rt.k, ctx.rt
        exact = rt.dtype == torch.float32            # the 32-bit path: the sublayers read x as it is
        h = x
        if not exact:
            left = ctx.shared.get(ROUNDED_STREAM)    # the block before left the rows it wrote, rounded
            h = left[1] if left is not None and left[0] is x else k.round_rows(x, ctx.ws.take(tuple(x.shape), rt.dtype))
        y = ctx.ws.take(tuple(x.shape), torch.float32)
        self._run(self.mixer, ctx, y, binding, h)
        h = None if exact else ctx.ws.take(tuple(x.shape), rt.dtype)
        k.sum_norm(y, self.alpha, self.norm1.gain, self.norm1.eps, self.norm1.kind, x, h)
        if self.feed_forward is not None:
            self._run(self.feed_forward, ctx, y, x if exact else h)
            k.sum_norm(y, self.alpha, self.norm2.gain, self.norm2.eps, self.norm2.kind, x, h)
        ctx.shared[ROUNDED_STREAM] = None if exact else (x, h)


class ParallelBlock(Block):
    """h = norm1(x); x += mixer(h) + feed_forward(h): one norm, and both sublayers read its output (a
    layer may have no feed-forward).  Each sublayer adds into the 32-bit stream in the epilogue of its
    last product."""
    graph_safe = True
    norm1_name = "norm1"

    def __init__(self, norm_factory, mixer, feed_forward, prefix):
        super().__init__(norm_factory, mixer, feed_forward, prefix)
        self.norm1 = norm_factory(self.norm1_name)

    def parts(self):
        return [p for p in (self.norm1, self.mixer, self.feed_forward) if p is not None]

    def tensors(self) -> List[TensorDecl]:
        return [d for p in self.parts() for d in p.tensors()]

    def load(self, store, rt) -> None:
        for part in self.parts():
            part.load(store, rt)

    def first_norm(self):
        return self.norm1

    def forward(self, ctx, binding: CacheBinding, x, normed=None, following=None) -> None:
        h = normed if normed is not None else self.norm1.forward(ctx, x)
        self.mixer.forward(ctx, binding, h, x)
        if self.feed_forward is not None:
            self.feed_forward.forward(ctx, h, x)


class SandwichNormBlock(Block):
    """x += norm1b(mixer(norm1(x))); x += norm2b(feed_forward(norm2(x))): a norm on each sublayer's input and one on its
    output (a layer may have no feed-forward, and then no second pair).  The outer norm and the sum are one 32-bit pass
    over the sublayer's 32-bit output (`Norm.add_to`: RMS norms and TanhNorm); where the norm that reads the sum is a
    TanhNorm that pass writes it too, the next block's first norm included."""
    graph_safe = True
    norm_names = ("norm1", "norm1b", "norm2", "norm2b")

    def __init__(self, norm_factory, mixer, feed_forward, prefix):
        super().__init__(norm_factory, mixer, feed_forward, prefix)
        names = self.norm_names if feed_forward is not None else self.norm_names[:2]
        self.norms = [norm_factory(name) for name in names]
        for norm in self.norms[1::2]:
            if not hasattr(norm, "add_to"):
                raise ConfigError(f"a norm on a sublayer's output adds it into the stream ({type(norm).__name__} cannot)")

    def parts(self):
        return [p for p in (*self.norms, self.mixer, self.feed_forward) if p is not None]

    def tensors(self) -> List[TensorDecl]:
        return [d for p in self.parts() for d in p.tensors()]

    def load(self, store, rt) -> None:
        for part in self.parts():
            part.load(store, rt)

    def first_norm(self):
        return self.norms[0]

    @staticmethod
    def following_of(ctx, part, norm, n_rows: int):
        """The norm behind a sum as work for the pass that makes the sum, whatever part's output it adds."""
        return norm.following_values(ctx, n_rows) if hasattr(norm, "following_values") else None

    _run = staticmethod(SublayerNormBlock._run)

    def forward(self, ctx, binding: CacheBinding, x, normed=None, following=None) -> None:
        h = normed if normed is not None else self.norms[0].forward(ctx, x)
        y = ctx.ws.take(tuple(x.shape), torch.float32)
        self._run(self.mixer, ctx, y, binding, h)
        if self.feed_forward is None:
            self.norms[1].add_to(ctx, y, x, following)
            return
        second = self.following_of(ctx, None, self.norms[2], x.shape[0])
        self.norms[1].add_to(ctx, y, x, second)
        h = second.values if second is not None else self.norms[2].forward(ctx, x)
        self._run(self.feed_forward, ctx, y, h)
        self.norms[3].add_to(ctx, y, x, following)


class ShiftedNorm(Norm):
    """A run's first norm with its token shift, bound to the state of that run (see `ScaledPreNormBlock`).  It offers itself to
    no product."""

    def __init__(self, block, state_index: int):
        super().__init__({}, block.prefix)
        self.norm, self.share, self.state_index = block.norm1, block.share, state_index

    def arguments(self, ctx):
        return self.share, ctx.cache.state(self.state_index), ctx.positions, ctx.seq_rows


class FollowingSum:
    """A norm handed to the block before: `values` get its rows in the pass that adds that block's last sublayer's output."""

    def __init__(self, norm, shift, values):
        self.norm, self.shift, self.values = norm, shift, values

    def arguments(self):
        return (self.norm.gain, self.norm.eps, self.values)


class ScaledPreNormBlock(Block):
    """x += m ls1 mixer(shift(norm1(x))); x += m ls2 feed_forward(norm2(x)): a layer scale (`layer_scale`: vectors `ls1`, `ls2`)
    and the residual's factor m (`residual_mult`) on each sublayer's output, and (`token_shift`: the vector `shift`) what the
    mixer reads moved towards the token before, h + (h' - h) shift with h' the previous token's h (zeros before the first), as
    it was before it was moved.  A layer may have no feed-forward (it then has no norm2 and no ls2).

    The outputs of a sublayer are stored as 32-bit rows and go into the stream in one 32-bit pass: a pair of mixers' two outputs
    with their norms or factors, the layer scale and m, the sum, and the norm behind it (the next block's first norm included:
    in steps of single tokens with its shift; else, since a shift reads the stream of the token before, that norm is a pass of
    its own).  h' is per-request state: two rows, the one behind position p in copy p & 1.

    The norms are RMS norms whose gains are kept 32-bit.  `residual_mult`, `layer_scale` and `token_shift` come with the norm's
    parameters."""
    graph_safe = True

    def __init__(self, norm_factory, mixer, feed_forward, prefix):
        super().__init__(norm_factory, mixer, feed_forward, prefix)
        self.norm1 = norm_factory("norm1")
        self.norm2 = norm_factory("norm2") if feed_forward is not None else None
        if getattr(self.norm1, "kind", None) != "rms":
            raise ConfigError("a norm with a token shift, or behind a scaled sum, is an RMS norm")
        for part in (mixer, feed_forward):
            if part is not None and not getattr(part, "stores_output", False) and getattr(type(part), "forward_apart", None) in (
                    None, Mixer.forward_apart):
                raise ConfigError(f"a sublayer whose output is scaled must be able to store it ({type(part).__name__} cannot)")
        p = self.norm1.params
        self.width, self.mult = int(p["size"]), float(p.get("residual_mult", 1.0))
        self.shift, self.layer_scale = bool(p.get("token_shift", False)), bool(p.get("layer_scale", False))
        self.share = None

    def parts(self):
        return [p for p in (self.norm1, self.mixer, self.norm2, self.feed_forward) if p is not None]

    def _vectors(self):
        scales = ["ls1"] + (["ls2"] if self.feed_forward is not None else []) if self.layer_scale else []
        return (["shift"] if self.shift else []), scales

    def tensors(self) -> List[TensorDecl]:
        shift, scales = self._vectors()
        return ([d for p in self.parts() for d in p.tensors()] + [TensorDecl(self.prefix + n, (self.width,), "bias") for n in shift]
                + [TensorDecl(self.prefix + n, (self.width,), "gain") for n in scales])

    def state_spec(self):
        return StateSpec(2 * self.width) if self.shift else None

    def load(self, store, rt) -> None:
        for part in self.parts():
            part.load(store, rt)
        for norm in (self.norm1, self.norm2):
            if norm is not None:
                norm.gain = norm.gain.float().contiguous()
        if self.shift:
            self.share = store.vector(self.prefix + "shift").float().contiguous()

        def scales_of(terms, name):
            # what a term is multiplied by, column by column: its own gain and factor, the layer scale, m
            ls = store.vector(self.prefix + name).float() if self.layer_scale else torch.ones(self.width, device=rt.device)
            return [((ls * (t.factor * self.mult) if t.gain is None else t.gain.float() * ls * (t.factor * self.mult)).contiguous(), t.norm_eps)
                    for t in terms]
        self.mixer_terms = scales_of(self.mixer.output_terms(), "ls1")
        self.ff_terms = scales_of([OutputTerm()], "ls2") if self.feed_forward is not None else None

    def first_norm(self):
        return self.norm1

    def entry_norm(self, binding: CacheBinding):
        return ShiftedNorm(self, binding.block_state) if self.shift else self.norm1

    def last_part(self):
        return self.feed_forward if self.feed_forward is not None else self.mixer

    @staticmethod
    def following_of(ctx, part, norm, n_rows: int):
        """The norm behind a sum as work for the pass that makes the sum."""
        if isinstance(norm, ShiftedNorm):
            if not ctx.decode_only:
                return None
            return FollowingSum(norm.norm, norm.arguments(ctx), ctx.ws.take((n_rows, norm.norm.size), ctx.rt.dtype))
        if getattr(norm, "kind", None) != "rms" or norm.gain is None or norm.gain.dtype != torch.float32:
            return None
        return FollowingSum(norm, None, ctx.ws.take((n_rows, norm.size), ctx.rt.dtype))

    def _add(self, ctx, outs, terms, x, following) -> None:
        ctx.rt.k.scaled_sum([(y, scales, eps) for y, (scales, eps) in zip(outs, terms)], x,
                            norm=None if following is None else following.arguments(),
                            shift=None if following is None else following.shift)

    def forward(self, ctx, binding: CacheBinding, x, normed=None, following=None) -> None:
        h = normed
        if h is None and self.shift:
            entry = self.entry_norm(binding)
            h = ctx.rt.k.shifted_norm(x, self.norm1.gain, self.norm1.eps, *entry.arguments(ctx), ctx.ws.take(tuple(x.shape), ctx.rt.dtype))
        elif h is None:
            h = self.norm1.forward(ctx, x)
        outs = [ctx.ws.take(tuple(x.shape), torch.float32) for _ in self.mixer_terms]
        self.mixer.forward_apart(ctx, binding, h, outs)
        if self.feed_forward is None:
            self._add(ctx, outs, self.mixer_terms, x, following)
            return
        second = self.following_of(ctx, None, self.norm2, x.shape[0])
        self._add(ctx, outs, self.mixer_terms, x, second)
        self.feed_forward.forward(ctx, second.values, outs[0], accumulate=False)
        self._add(ctx, outs[:1], self.ff_terms, x, following)


register_block("prenorm", PreNormBlock)
register_block("prenorm_scaled", ScaledPreNormBlock)
register_block("sandwich_norm", SandwichNormBlock)
register_block("parallel", ParallelBlock)
register_block("prenorm_short_names", ShortNamedPreNormBlock)
register_block("sublayer_norm", SublayerNormBlock)
register_block("postnorm", PostNormBlock)
