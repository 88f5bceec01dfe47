"""The Lilunex decoder's configuration: config.json to a ModelSpec.

config.json names the design in `architecture` and gives `vocab`, `width`, `norm.eps`, `embedding.scale` and a list
`layers`.  Every layer has a `type` (which mixer), the mixer's sizes (`mixer`) and its feed-forward (`mlp`, or null
for none):

* "wkv": time mixing with a state matrix a head, decayed per key channel (`heads`, `dim`); the rank of its decay's
  low-rank product is the first dimension of the tensor `mix.w1`;
* "attention": grouped-query attention with biases (`heads`, `kv_heads`, `dim`, `vdim`, `scale`), queries and keys
  normed over all their rows at once, the first `rot.dims` places of a head rotated in half-apart pairs (`rot.base`, the
  frequencies divided by `rot.scaling.factor`), a sliding window of `mask.size` positions beside the first
  `mask.keep_first` ones, and a sink a head in the softmax; with `kv_from` it reads that layer's keys and values;
* "delta": the gated delta rule behind short convolutions (`heads`, `kv_heads`, `dim`, `vdim`, `conv`);
* `mlp` {"kind": "dense", "ff"}: two matrices and the square of relu; {"kind": "moe"}: `router.experts` gated units of
  `expert.ff` and `router.identity` identities, of which a token takes the `router.top` with the largest softmax scores
  plus a stored correction, weighted by the scores over their sum; `shared` (`ff`): one more unit for every token, times
  the sigmoid of a logit of its own.

A layer is x += norm1b(mixer(norm1(x))); x += norm2b(mlp(norm2(x))) with norms tanh(alpha x) w + b.  Layer i's tensors
start with `l<i>.`; beside them there are `embed` (its rows times the scale), `final.norm` and `head`.
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


class LilunexConfig(ModelConfig):
    architecture = "Lilunex"
    model_type = "lilunex"

    def __init__(self, cfg: Dict[str, Any], ranks: Optional[Dict[int, int]] = None):
        if not isinstance(cfg, dict):
            raise ConfigError("config.json is not a JSON object")
        self.cfg = copy.deepcopy(cfg)
        self.width = get_whole(cfg, "width")
        self.vocab = get_whole(cfg, "vocab")
        self.eps = get_number(_object(cfg, "norm", ""), "eps")
        self.embedding_scale = get_number(_object(cfg, "embedding", "", optional=True) or {}, "scale", 1.0, positive=False)
        self.ranks = dict(ranks or {})            # of the wkv layers, where the checkpoint's tensors told
        layers = cfg.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json layers is not a list of layers")
        for i, entry in enumerate(layers):
            if not isinstance(entry, dict):
                raise ConfigError(f"config.json layers[{i}] is not an object")
        self.kv_from: List[Optional[int]] = [self._kv_from(layers, i) for i in range(len(layers))]
        self.layers: List[Dict[str, Any]] = []
        for i, entry in enumerate(layers):
            where = f"layers[{i}]."
            self.layers.append({"mixer": self._mixer(i, entry.get("type"), _object(entry, "mixer", where), where),
                                "mlp": self._mlp(entry.get("mlp"), where)})

    # ------------------------------------------------------------------ the parts of a layer
    @staticmethod
    def _kv_from(layers, i: int) -> Optional[int]:
        mixer = layers[i].get("mixer")
        if layers[i].get("type") != "attention" or not isinstance(mixer, dict) or mixer.get("kv_from") is None:
            return None
        where = f"layers[{i}].mixer.kv_from"
        j = get_whole(mixer, "kv_from", minimum=0)
        if j >= i or layers[j].get("type") != "attention":
            raise ConfigError(f"config.json {where} = {j} is not an attention layer before it")
        other = layers[j].get("mixer") or {}
        if other.get("kv_from") is not None:
            raise ConfigError(f"config.json {where} = {j}: that layer has no keys and values of its own")
        for key in ("kv_heads", "dim", "vdim"):
            if other.get(key) != mixer.get(key):
                raise ConfigError(f"config.json {where} = {j}: its {key} {other.get(key)} is not this layer's {mixer.get(key)}")
        return j

    def _mixer(self, i: int, kind, mixer: Dict[str, Any], where: str) -> PartSpec:
        common = {"hidden_size": self.width, "eps": self.eps}
        if kind == "wkv":
            return PartSpec("time_mix", {**common, "heads": get_whole(mixer, "heads"), "dim": get_whole(mixer, "dim"),
                                         "rank": self.ranks.get(i, self._usual_rank())})
        if kind == "delta":
            return PartSpec("gated_delta_rule", {**common, "heads": get_whole(mixer, "heads"), "kv_heads": get_whole(mixer, "kv_heads"),
                                                 "dim": get_whole(mixer, "dim"), "vdim": get_whole(mixer, "vdim"),
                                                 "conv": get_whole(mixer, "conv")})
        if kind != "attention":
            raise ConfigError(f"config.json {where}type = {kind!r} is not a mixer of this design (wkv, attention, delta)")
        where += "mixer."
        mask, rot = _object(mixer, "mask", where, optional=True), _object(mixer, "rot", where, optional=True)
        position = None
        if rot is not None and get_whole(rot, "dims", minimum=0) > 0:
            scaling = _object(rot, "scaling", where + "rot.", optional=True)
            position = PartSpec("rope", {
                "head_dim": get_whole(mixer, "dim"), "rotary_dim": get_whole(rot, "dims", minimum=2), "theta": get_number(rot, "base"),
                "pairing": "halves",
                "scaling": None if scaling is None else {"kind": "linear", "factor": get_number(scaling, "factor")}})
        return PartSpec("masked_attention", {
            **common, "heads": get_whole(mixer, "heads"), "kv_heads": get_whole(mixer, "kv_heads"), "dim": get_whole(mixer, "dim"),
            "vdim": get_whole(mixer, "vdim"), "scale": get_number(mixer, "scale"), "bias": True, "out_bias": True, "qk_norm": "rows",
            "sink": "heads", "reads_cache": self.kv_from[i] is not None, "position": position,
            "mask": None if mask is None else {"kind": "window", "size": get_whole(mask, "size"),
                                               "keep": get_whole(mask, "keep_first", 0, minimum=0)}})

    def _usual_rank(self) -> int:
        """The rank of a decay's low-rank product where no tensor tells it (random weights): about a thirty-second of
        the width, in sixteens."""
        return max(16, self.width // 512 * 16)

    def _mlp(self, mlp, where: str) -> Optional[PartSpec]:
        if mlp is None:
            return None
        if not isinstance(mlp, dict):
            raise ConfigError(f"config.json {where}mlp = {mlp!r} is not an object")
        if mlp.get("kind") == "dense":
            return PartSpec("dense_mlp", {"hidden_size": self.width, "ff": get_whole(mlp, "ff"), "activation": "relu_squared"})
        if mlp.get("kind") != "moe":
            raise ConfigError(f"config.json {where}mlp.kind = {mlp.get('kind')!r} is not a feed-forward of this design (dense, moe)")
        expert, router = _object(mlp, "expert", where + "mlp."), _object(mlp, "router", where + "mlp.")
        shared = _object(mlp, "shared", where + "mlp.", optional=True)
        return PartSpec("routed_experts", {
            "hidden_size": self.width, "experts": get_whole(router, "experts"), "identity": get_whole(router, "identity", 0, minimum=0),
            "top": get_whole(router, "top"), "ff": get_whole(expert, "ff"), "limit": None, "alpha": 1.0, "shift": 0.0,
            "router": {"scores": "softmax_all", "correction": True},
            "shared": None if shared is None else {"ff": get_whole(shared, "ff"), "unit": "gated", "gate": "sg"}})

    @classmethod
    def from_dict(cls, cfg: Dict[str, Any]) -> "LilunexConfig":
        return cls(cfg)

    def to_dict(self) -> Dict[str, Any]:
        return copy.deepcopy(self.cfg)

    # ------------------------------------------------------------------ sizes that only tensors tell
    def _rank_tensors(self) -> Dict[str, int]:
        return {f"l{i}.mix.w1": i for i, layer in enumerate(self.layers) if layer["mixer"].kind == "time_mix"}

    def size_tensors(self) -> List[str]:
        return list(self._rank_tensors())

    def with_sizes(self, shapes: Dict[str, tuple]) -> "LilunexConfig":
        of = self._rank_tensors()
        return LilunexConfig(self.cfg, {of[name]: int(shape[0]) for name, shape in shapes.items() if len(shape) == 2 and shape[0] > 0})

    # ------------------------------------------------------------------ the model as data
    def model_spec(self) -> ModelSpec:
        norm = PartSpec("tanh_norm", {"size": self.width})
        layers = [LayerSpec(block="sandwich_norm", mixer=layer["mixer"], feed_forward=layer["mlp"], norm=norm, prefix=f"l{i}.")
                  for i, layer in enumerate(self.layers)]
        order = [Run(layer=i, cache=i if j is None else j, writes_cache=j is None) for i, j in enumerate(self.kv_from)]
        return ModelSpec(
            hidden_size=self.width, vocab_size=self.vocab,
            embedding=PartSpec("token_embedding", {"vocab_size": self.vocab, "hidden_size": self.width, "tensor": "embed",
                                                   "scale": self.embedding_scale}),
            layers=layers, order=order, final_norm=PartSpec("tanh_norm", {"size": self.width, "tensor": "final.norm"}),
            head=PartSpec("lm_head", {"vocab_size": self.vocab, "hidden_size": self.width, "tensor": "head"}),
            max_positions=UNBOUNDED_POSITIONS)
