"""A decoder model put together from a `ModelSpec`: embedding, blocks in their execution
order, final norm and head.  It knows no architecture: the configuration decided the parts.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Tuple

import torch

from ..cache.manager import GroupPlan
from ..config.base import ConfigError, ModelConfig
from ..parts.base import ROUNDED_STREAM, CacheBinding, TensorDecl, build_block, build_part


@dataclass
class CachePlan:
    """What the model's runs need from the cache manager: for each group its need and number
    of storing runs; for each run its binding; the sizes of the state arenas."""
    group_specs: List
    group_layers: List[int]
    bindings: List[CacheBinding]
    state_elems: List[tuple]


class DecoderModel:
    def __init__(self, config: ModelConfig):
        self.config = config
        spec = config.model_spec()
        self.spec = spec
        self.hidden_size = spec.hidden_size
        self.vocab_size = spec.vocab_size
        self.max_positions = spec.max_positions
        self.embedding = build_part("embedding", spec.embedding)
        self.blocks = []
        for layer in spec.layers:
            mixer = build_part("mixer", layer.mixer, layer.prefix)
            # a layer may have no feed-forward (its block then has to be one that takes none)
            ffn = build_part("feed_forward", layer.feed_forward, layer.prefix) if layer.feed_forward is not None else None
            self.blocks.append(build_block(layer.block, layer.norm, mixer, ffn, layer.prefix))
        # rewrites of the residual stream that runs may enter through (they read the embedding's output)
        self.entries = [build_part("stream", e) for e in spec.entries]
        self.final_norm = build_part("norm", spec.final_norm)
        self.head = build_part("head", spec.head)
        self.order = list(spec.order)
        for run in self.order:
            if not 0 <= run.layer < len(self.blocks):
                raise ConfigError(f"the execution order names layer {run.layer}, the model has {len(self.blocks)}")
            if run.enter is not None and not 0 <= run.enter < len(self.entries):
                raise ConfigError(f"a run enters through entry {run.enter}, the model has {len(self.entries)}")
        self.cache_plan = self._plan_cache()

    # ------------------------------------------------------------------ declarations
    def tensors(self) -> List[TensorDecl]:
        out = list(self.embedding.tensors())
        for e in self.entries:
            out += e.tensors()
        for b in self.blocks:
            out += b.tensors()
        return out + self.final_norm.tensors() + self.head.tensors()

    def _plan_cache(self) -> CachePlan:
        group_of_key: Dict[Tuple, int] = {}
        specs, counts = [], []
        where: Dict[int, Tuple[int, int]] = {}      # cache id -> (group, index in group)
        needs: Dict[int, object] = {}               # cache id -> what its writer and its readers need of it
        for run in self.order:                      # first the runs that store
            cs = self.blocks[run.layer].mixer.cache_spec()
            if cs is None or not run.writes_cache:
                continue
            if run.cache in needs:
                raise ConfigError(f"two runs store into cache {run.cache}")
            needs[run.cache] = cs
        for run in self.order:                      # then those that only read
            cs = self.blocks[run.layer].mixer.cache_spec()
            if cs is None or run.writes_cache:
                continue
            if run.cache not in needs:
                raise ConfigError(f"a run of layer {run.layer} reads cache {run.cache}, which no run stores")
            if needs[run.cache].shape_key() != cs.shape_key():
                raise ConfigError(f"layer {run.layer} cannot read cache {run.cache}: its shape differs")
            needs[run.cache] = needs[run.cache].widened(cs)
        for cache, cs in needs.items():
            g = group_of_key.setdefault(cs.group_key(), len(specs))
            if g == len(specs):
                specs.append(cs)
                counts.append(0)
            where[cache] = (g, counts[g])
            counts[g] += 1
        bindings, state_elems = [], []

        def arena(spec) -> int:
            state_elems.append((spec.elems, spec.dtype))
            return len(state_elems) - 1

        for run in self.order:
            block = self.blocks[run.layer]
            mixer, own = block.mixer, block.state_spec()
            cs = mixer.cache_spec()
            b = CacheBinding(writes=run.writes_cache)
            if cs is not None:
                b.group, b.index = where[run.cache]
            states = [arena(ss) for ss in mixer.state_specs()]
            if states:
                b.state_index, b.more_states = states[0], tuple(states[1:])
            if own is not None:
                b.block_state = arena(own)
            bindings.append(b)
        if self.embedding.state_spec() is not None:
            self.embedding.state_index = arena(self.embedding.state_spec())
        return CachePlan(specs, counts, bindings, state_elems)

    def group_plans(self, page_size: int, pages_of_group) -> List[GroupPlan]:
        """`pages_of_group(spec, n_layers, page_size)` decides each pool's size."""
        return [GroupPlan(s, n, page_size, pages_of_group(s, n, page_size))
                for s, n in zip(self.cache_plan.group_specs, self.cache_plan.group_layers)]

    # ------------------------------------------------------------------ weights
    def load(self, store, rt) -> None:
        self.embedding.load(store, rt)
        for e in self.entries:
            e.load(store, rt)
        for b in self.blocks:
            b.load(store, rt)
        self.final_norm.load(store, rt)
        self.head.load(store, rt)
        # a head tied to the embedding may keep the matrix in a form of its own (repacked for its
        # product): the head says so, the embedding then reads that copy and the other is dropped
        if self.head.shares_with(self.embedding):
            self.embedding.read_from(self.head, store)

    # ------------------------------------------------------------------ the step
    def embed(self, ctx, out=None) -> torch.Tensor:
        """The residual stream before the first run: float32 [T, hidden] (into `out` if given)."""
        x = self.embedding.forward(ctx, out=out)
        if self.entries:
            # kept for the runs that enter through a rewrite of the stream; x itself moves on
            x0 = ctx.ws.take(tuple(x.shape), torch.float32)
            x0.copy_(x)
            ctx.shared["embedding_output"] = x0
        return x

    def forward(self, ctx) -> torch.Tensor:
        """The residual stream after every run: float32 [T, hidden]."""
        x = self.embed(ctx)
        self.forward_runs(ctx, x, 0, len(self.order))
        return x

    def forward_runs(self, ctx, x: torch.Tensor, first: int, end: int) -> None:
        """Runs first .. end - 1 of the execution order on the residual stream x, in place."""
        normed = None        # the next block's first norm, where the block before it did its work
        for i in range(first, end):
            run, binding = self.order[i], self.cache_plan.bindings[i]
            block = self.blocks[run.layer]
            if run.enter is not None:
                self.entries[run.enter].forward(ctx, x, ctx.shared["embedding_output"])
                ctx.shared[ROUNDED_STREAM] = None        # what a block left of the stream it wrote is no longer the stream
            following = None
            if i + 1 < end and self.order[i + 1].enter is None:     # a rewritten stream is normed by its own pass
                after = self.blocks[self.order[i + 1].layer]
                following = block.following_of(ctx, block.last_part(), after.entry_norm(self.cache_plan.bindings[i + 1]), x.shape[0])
            if normed is None and following is None:
                block.forward(ctx, binding, x)          # a block that knows nothing of this is called plainly
            else:
                block.forward(ctx, binding, x, normed, following)
            normed = None if following is None else following.values

    def run_is_graph_safe(self, i: int) -> bool:
        """Whether run i's block and its parts are all fixed launch sequences (see Part.graph_safe)."""
        block = self.blocks[self.order[i].layer]
        entry = self.order[i].enter
        parts = (block, block.mixer, block.feed_forward, None if entry is None else self.entries[entry])
        return all(getattr(p, "graph_safe", False) for p in parts if p is not None)

    def ends_are_graph_safe(self) -> bool:
        """Whether what runs before the first run and behind the last (`embed`, `logits`) is a fixed
        launch sequence too, so that it can be captured with the runs beside it."""
        return all(getattr(p, "graph_safe", False) for p in (self.embedding, self.final_norm, self.head))

    def logits(self, ctx, x: torch.Tensor, rows: torch.Tensor, out=None) -> torch.Tensor:
        """Final norm and head at the rows asked for: float32 [len(rows), vocab]."""
        h = self.final_norm.forward(ctx, x, rows=rows)
        return self.head.forward(ctx, h, out)
