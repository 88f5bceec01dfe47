"""The Bafavik decoder's configuration: config.json to a ModelSpec.

config.json names the design in `architecture` and gives `vocab`, `width`, `norm.eps`, `residual_mult`, `logit_scale`,
`embedding` (`scale` and, optionally, `bigram`: `buckets`, `mul_prev`, `mul_cur`), a list `layers` and, optionally, `loop`.
Every layer has a `type` (which mixer), the mixer's sizes (`mixer`) and its feed-forward (`mlp`: {"kind": "dense", "ff"}, or
null for none):

* "parallel": `left_scale` times attention plus `right_scale` times linear attention.  `left`: grouped-query attention with
  biases on every projection (`heads`, `kv_heads`, `dim`, `vdim`, `scale`), the first `rot.dims` places of a head rotated in
  half-apart pairs (`rot.base`), queries and keys then of root mean square 1 a head.  `right`: linear attention with a
  constant decay a head (`heads`, `dim`, `vdim`, `decay`);
* "attention": differential attention without rotation (`heads`, `kv_heads`, `dim`, `vdim`, `scale`, `diff`), biases on q, k
  and v, chunks of `mask.size` positions, a sigmoid gate on the heads;
* "parallel_2": half the sum of two outputs, each RMS-normed over the width with a gain.  `left`: attention behind short
  convolutions of `conv` taps (`heads`, `kv_heads`, `dim`, `vdim`, `scale`), neighbouring places rotated, a sigmoid gate on the
  heads.  `right`: the gated delta rule (`heads`, `kv_heads`, `dim`, `vdim`, `conv`) with a decay a head and key channel and a
  sigmoid gate, both of low rank: the ranks are the first dimensions of the tensors `mix.right.a1` and `mix.right.g1`.

A layer is x += m ls1 mixer(shift(norm1(x))); x += m ls2 down(relu(up(norm2(x)))^2) with RMS norms whose gains are stored
around zero (1 + w), layer scales `ls1` and `ls2`, m the `residual_mult`, and what the mixer reads moved towards the token
before by `shift`, column by column.  `loop` = {start, stop, times}: layers start .. stop - 1 run `times` times in a row with
the same tensors, each pass with caches and states of its own.  Layer i's tensors start with `l<i>.`; beside them there are
`embed`, `bigram`, `final.norm` and `head` (logits = head norm(x) logit_scale).
"""
from __future__ import annotations

import copy
from typing import Any, Dict, List, Optional

from .base import ConfigError, LayerSpec, ModelConfig, ModelSpec, PartSpec, Run, get_number, get_whole

# the design leaves positions unbounded; the engine sizes its block tables by this unless told otherwise
UNBOUNDED_POSITIONS = 1 << 20


def _object(cfg: Dict[str, Any], key: str, where: str, optional: bool = False) -> Optional[Dict[str, Any]]:
    v = cfg.get(key)
    if v is None and optional:
        return None
    if not isinstance(v, dict):
        raise ConfigError(f"config.json {where}{key} = {v!r} is not an object")
    return v


class BafavikConfig(ModelConfig):
    architecture = "Bafavik"
    model_type = "bafavik"

    def __init__(self, cfg: Dict[str, Any], ranks: Optional[Dict[str, int]] = None):
        if not isinstance(cfg, dict):
            raise ConfigError("config.json is not a JSON object")
        self.cfg = copy.deepcopy(cfg)
        self.width = get_whole(cfg, "width")
        self.vocab = get_whole(cfg, "vocab")
        self.eps = get_number(_object(cfg, "norm", ""), "eps")
        self.residual_mult = get_number(cfg, "residual_mult", 1.0, positive=False)
        self.logit_scale = get_number(cfg, "logit_scale", 1.0, positive=False)
        embedding = _object(cfg, "embedding", "", optional=True) or {}
        self.embedding_scale = get_number(embedding, "scale", 1.0, positive=False)
        bigram = _object(embedding, "bigram", "embedding.", optional=True)
        self.pairs = None if bigram is None else {"tensor": "bigram", "buckets": get_whole(bigram, "buckets"),
                                                  "mul_prev": get_whole(bigram, "mul_prev", minimum=0),
                                                  "mul_cur": get_whole(bigram, "mul_cur", minimum=0)}
        self.ranks = dict(ranks or {})            # of the low-rank products, by tensor, where the checkpoint's tensors told
        layers = cfg.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json layers is not a list of layers")
        self.layers: List[Dict[str, Any]] = []
        for i, entry in enumerate(layers):
            where = f"layers[{i}]."
            if not isinstance(entry, dict):
                raise ConfigError(f"config.json layers[{i}] is not an object")
            self.layers.append({"mixer": self._mixer(i, entry.get("type"), _object(entry, "mixer", where), where + "mixer."),
                                "mlp": self._mlp(entry.get("mlp"), where)})
        loop = _object(cfg, "loop", "", optional=True)
        self.loop = None
        if loop is not None:
            start, stop = get_whole(loop, "start", minimum=0), get_whole(loop, "stop", minimum=0)
            times = get_whole(loop, "times", minimum=0)
            if not start <= stop <= len(layers):
                raise ConfigError(f"config.json loop: layers {start} .. {stop} - 1 of {len(layers)}")
            self.loop = (start, stop, times)

    # ------------------------------------------------------------------ the parts of a layer
    def _heads(self, mixer: Dict[str, Any]) -> Dict[str, Any]:
        return {"hidden_size": self.width, "heads": get_whole(mixer, "heads"), "kv_heads": get_whole(mixer, "kv_heads"),
                "dim": get_whole(mixer, "dim"), "vdim": get_whole(mixer, "vdim"), "scale": get_number(mixer, "scale"), "eps": self.eps}

    @staticmethod
    def _rotation(mixer: Dict[str, Any], where: str, pairing: str) -> Optional[PartSpec]:
        rot = _object(mixer, "rot", where, optional=True)
        if rot is None or get_whole(rot, "dims", minimum=0) == 0:
            return None
        return PartSpec("rope", {"head_dim": get_whole(mixer, "dim"), "rotary_dim": get_whole(rot, "dims", minimum=2),
                                 "theta": get_number(rot, "base"), "pairing": pairing})

    def _mixer(self, i: int, kind, mixer: Dict[str, Any], where: str) -> PartSpec:
        if kind == "attention":
            mask = _object(mixer, "mask", where, optional=True)
            return PartSpec("masked_attention", {
                **self._heads(mixer), "maps": 2, "diff": get_number(mixer, "diff", positive=False), "bias": True, "gate": "elements",
                "mask": None if mask is None else {"kind": "chunk", "size": get_whole(mask, "size")}, "position": None})
        if kind not in ("parallel", "parallel_2"):
            raise ConfigError(f"config.json {where[:-6]}type = {kind!r} is not a mixer of this design (parallel, attention, parallel_2)")
        left, right = _object(mixer, "left", where), _object(mixer, "right", where)
        common = {"hidden_size": self.width, "eps": self.eps}
        if kind == "parallel":
            attention = PartSpec("masked_attention", {
                **self._heads(left), "bias": True, "out_bias": True, "qk_norm": "plain",
                "position": self._rotation(left, where + "left.", "halves"), "names": {"scope": "mix.left."}})
            decay = right.get("decay")
            if not isinstance(decay, list) or any(isinstance(d, bool) or not isinstance(d, (int, float)) for d in decay):
                raise ConfigError(f"config.json {where}right.decay = {decay!r} is not a list of numbers")
            linear = PartSpec("lightning_attention", {
                **common, "heads": get_whole(right, "heads"), "dim": get_whole(right, "dim"), "vdim": get_whole(right, "vdim"),
                "decay": [float(d) for d in decay], "names": {"scope": "mix.right."}})
            if len(decay) != get_whole(right, "heads"):
                raise ConfigError(f"config.json {where}right.decay has {len(decay)} numbers for {get_whole(right, 'heads')} heads")
            return PartSpec("paired_mixers", {
                **common, "combine": "scaled", "left": attention, "right": linear,
                "scales": [get_number(mixer, "left_scale", 1.0, positive=False), get_number(mixer, "right_scale", 1.0, positive=False)]})
        attention = PartSpec("masked_attention", {
            **self._heads(left), "conv": get_whole(left, "conv"), "gate": "elements",
            "position": self._rotation(left, where + "left.", "neighbours"), "names": {"scope": "mix.left."}})
        rank = lambda name: {"rank": self.ranks.get(f"l{i}.mix.right.{name}", self._usual_rank())}
        delta = PartSpec("gated_delta_rule", {
            **common, "heads": get_whole(right, "heads"), "kv_heads": get_whole(right, "kv_heads"), "dim": get_whole(right, "dim"),
            "vdim": get_whole(right, "vdim"), "conv": get_whole(right, "conv"), "decay": rank("a1"), "gate": rank("g1"),
            "gate_act": "sigmoid", "names": {"scope": "mix.right."}})
        return PartSpec("paired_mixers", {**common, "combine": "normed", "mult": 0.5, "left": attention, "right": delta})

    def _usual_rank(self) -> int:
        """The rank of a low-rank product where no tensor tells it (random weights): about a thirty-second of the width, in
        sixteens."""
        return max(16, self.width // 512 * 16)

    def _mlp(self, mlp, where: str) -> Optional[PartSpec]:
        if mlp is None:
            return None
        if not isinstance(mlp, dict):
            raise ConfigError(f"config.json {where}mlp = {mlp!r} is not an object")
        if mlp.get("kind") != "dense":
            raise ConfigError(f"config.json {where}mlp.kind = {mlp.get('kind')!r} is not a feed-forward of this design (dense)")
        return PartSpec("dense_mlp", {"hidden_size": self.width, "ff": get_whole(mlp, "ff"), "activation": "relu_squared"})

    @classmethod
    def from_dict(cls, cfg: Dict[str, Any]) -> "BafavikConfig":
        return cls(cfg)

    def to_dict(self) -> Dict[str, Any]:
        return copy.deepcopy(self.cfg)

    # ------------------------------------------------------------------ sizes that only tensors tell
    def size_tensors(self) -> List[str]:
        return [f"l{i}.mix.right.{name}" for i, layer in enumerate(self.cfg["layers"]) if layer["type"] == "parallel_2" for name in ("a1", "g1")]

    def with_sizes(self, shapes: Dict[str, tuple]) -> "BafavikConfig":
        return BafavikConfig(self.cfg, {name: int(shape[0]) for name, shape in shapes.items() if len(shape) == 2 and shape[0] > 0})

    # ------------------------------------------------------------------ the model as data
    def run_order(self) -> List[int]:
        """The layers in the order they run."""
        n = len(self.layers)
        if self.loop is None:
            return list(range(n))
        start, stop, times = self.loop
        return list(range(start)) + list(range(start, stop)) * times + list(range(stop, n))

    def model_spec(self) -> ModelSpec:
        norm = PartSpec("rmsnorm", {"size": self.width, "eps": self.eps, "offset": 1.0, "residual_mult": self.residual_mult,
                                    "layer_scale": True, "token_shift": True})
        layers = [LayerSpec(block="prenorm_scaled", mixer=layer["mixer"], feed_forward=layer["mlp"], norm=norm, prefix=f"l{i}.")
                  for i, layer in enumerate(self.layers)]
        embedding = {"vocab_size": self.vocab, "hidden_size": self.width, "tensor": "embed", "scale": self.embedding_scale}
        if self.pairs is not None:
            embedding["pairs"] = self.pairs
        return ModelSpec(
            hidden_size=self.width, vocab_size=self.vocab,
            embedding=PartSpec("token_embedding" if self.pairs is None else "pair_embedding", embedding), layers=layers,
            # every run has a cache and a state of its own: a layer of the loop keeps one per pass
            order=[Run(layer=i, cache=at) for at, i in enumerate(self.run_order())],
            final_norm=PartSpec("rmsnorm", {"size": self.width, "eps": self.eps, "tensor": "final.norm", "offset": 1.0}),
            head=PartSpec("lm_head", {"vocab_size": self.vocab, "hidden_size": self.width, "tensor": "head", "scale": self.logit_scale}),
            max_positions=UNBOUNDED_POSITIONS)
