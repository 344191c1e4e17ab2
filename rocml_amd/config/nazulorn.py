"""Typed configuration of the Nazulorn decoder, read from config.json.

A Nazulorn layer works on several copies of the residual stream (hyper-connections): a sublayer reads the norm of a weighted
sum of the copies, and behind it every copy is formed anew from all the old ones and the sublayer's output.  The copies start equal
to the embedding's output; the model's output reads their sum.  A layer's mixer is

* **differential attention** (``type: attention``): two softmax maps per head over the same values, under a window, with rotated
  q and k; the second map counts against the first with one weight per layer, and every head's output is divided by its
  root mean square and multiplied by ``1 - diff``; or
* **gated linear attention** (``type: gla``): a matrix state per head with a decay per token and key channel, every head's
  output normed with one gain for all heads and gated by ``silu(W_g h)``.

The feed-forward is a mixture of small experts (softmax scores over all, a correction added for the choice only, weights times a
factor), of which the last few are identity experts that hand their input on, with a shared expert beside them; gate and up values
are held under a limit, ``g sigmoid(1.702 g) (u + 1)``.  It may be absent.  config.json gives every size layer by layer:

* ``architecture``: ``"Nazulorn"``; ``vocab``, ``width``, ``streams``; ``norm.eps``; ``embedding.scale``; ``residual_mult``;
  ``logit_scale``; ``max_positions`` or absent;
* ``layers[i]``: ``type``; for ``attention`` ``mixer`` has ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``diff``, ``mask.size`` (or no mask:
  everything before the query is seen) and ``rot`` (``base``, ``dims``, ``scaling`` with ``factor``, ``original``, ``fast``, ``slow`` or absent); for
  ``gla`` ``heads``, ``dim``, ``vdim`` and ``tau``;
  ``mlp``: null or ``{"kind": "moe", "expert": {"ff", "limit"}, "router": {"experts", "identity", "top", "scale"},
  "shared": {"ff", "limit"} or null}``.

The inner width of the decay's two small matrices is read from the checkpoint's tensor shapes (``with_shapes``); here it is the
configuration's ``mixer.decay_rank`` when given.

Constants the design fixes live here: the 1.702 in the experts' gate, the one added to their up values, the 1e-20 under the
experts' weights.
"""
from __future__ import annotations

import copy
import math
from dataclasses import dataclass, replace
from typing import Dict, List, Optional, Tuple

from ..errors import ConfigError, UnsupportedArchitectureError
from .spec import (BlockSpec, DifferentialAttentionSpec, GatedLinearAttentionSpec, ModelSpec, NormSpec, RopeSpec, RopeStretch,
                   RoutedExpertsSpec, default_schedule)

ARCHITECTURE = "Nazulorn"
EXPERT_ACTIVATION = "sigmoid_1702"
EXPERT_UP_OFFSET = 1.0
EXPERT_SUM_EPS = 1e-20
DEFAULT_DECAY_RANK = 16          # used for random models when the configuration names none
UNBOUNDED_POSITIONS = 1 << 30    # a model that names no limit


def _table(where: str, d: Dict, key: str) -> Dict:
    if not isinstance(d.get(key), dict):
        raise ConfigError(f"config.json lacks the table {where}{key}")
    return d[key]


def _int(where: str, d: Dict, key: str, least: int = 1) -> int:
    if key not in d:
        raise ConfigError(f"config.json lacks {where}{key!r}")
    v = d[key]
    if isinstance(v, bool) or not isinstance(v, int) or v < least:
        raise ConfigError(f"config.json {where}{key!r} must be an integer of at least {least}, found {v!r}")
    return v


def _num(where: str, d: Dict, key: str, positive: bool = True) -> float:
    if key not in d:
        raise ConfigError(f"config.json lacks {where}{key!r}")
    v = d[key]
    if isinstance(v, bool) or not isinstance(v, (int, float)) or not math.isfinite(v) or (positive and v <= 0):
        raise ConfigError(f"config.json {where}{key!r} must be a {'positive ' if positive else ''}number, found {v!r}")
    return float(v)


def _check_rot(where: str, m: Dict) -> None:
    if m.get("rot") is None:
        return
    rot = _table(where, m, "rot")
    base = _num(where + "rot.", rot, "base")
    dims = _int(where + "rot.", rot, "dims")
    if dims % 2 != 0 or dims > m["dim"]:
        raise ConfigError(f"config.json {where}rot.dims must be even and at most the head size {m['dim']}, found {dims}")
    if rot.get("scaling") is not None:
        sc = _table(where + "rot.", rot, "scaling")
        for key in ("factor", "original", "fast", "slow"):
            _num(where + "rot.scaling.", sc, key)
        if base <= 1:
            raise ConfigError(f"config.json {where}rot.base must be above 1 for a scaling, found {base}")


def _check_expert(where: str, d: Dict) -> None:
    _int(where, d, "ff")
    if d.get("limit") is not None:
        _num(where, d, "limit")


def _check_mlp(where: str, mlp) -> None:
    if mlp is None:
        return
    if not isinstance(mlp, dict) or mlp.get("kind") != "moe":
        raise ConfigError(f"config.json {where}mlp must be null or of kind 'moe', found {mlp!r}")
    w = where + "mlp."
    _check_expert(w + "expert.", _table(w, mlp, "expert"))
    r = _table(w, mlp, "router")
    experts, top = _int(w + "router.", r, "experts"), _int(w + "router.", r, "top")
    identity = _int(w + "router.", r, "identity", 0) if r.get("identity") is not None else 0
    if top > experts + identity:
        raise ConfigError(f"config.json {w}router: top {top} exceeds the {experts} experts and {identity} identity experts")
    if r.get("scale") is not None:
        _num(w + "router.", r, "scale", positive=False)
    if mlp.get("shared") is not None:
        _check_expert(w + "shared.", _table(w, mlp, "shared"))


def _check_layer(i: int, layer) -> Dict:
    where = f"layers[{i}]."
    kind = layer.get("type") if isinstance(layer, dict) else None
    if kind not in ("attention", "gla"):
        raise ConfigError(f"config.json {where}type is {kind!r}; known: attention, gla")
    m = _table(where, layer, "mixer")
    w = where + "mixer."
    for key in ("heads", "dim", "vdim"):
        _int(w, m, key)
    if kind == "attention":
        if m["heads"] % _int(w, m, "kv_heads") != 0:
            raise ConfigError(f"config.json {w[:-1]}: {m['heads']} heads are not a multiple of {m['kv_heads']} kv_heads")
        _num(w, m, "scale")
        _num(w, m, "diff", positive=False)
        if m.get("mask") is not None:
            mask = _table(w, m, "mask")
            if mask.get("size") is not None:
                _int(w + "mask.", mask, "size")
        _check_rot(w, m)
    else:
        _num(w, m, "tau")
        if m.get("decay_rank") is not None:
            _int(w, m, "decay_rank")
    _check_mlp(where, layer.get("mlp"))
    return copy.deepcopy(layer)


@dataclass(frozen=True)
class NazulornConfig:
    vocab: int
    width: int
    streams: int
    eps: float
    embedding_scale: float
    residual_mult: float
    logit_scale: float
    layers: Tuple[Dict, ...]               # as config.json has them, validated
    max_positions: Optional[int] = None
    eos_token_id: Optional[Tuple[int, ...]] = None

    @classmethod
    def from_dict(cls, raw: Dict) -> "NazulornConfig":
        if raw.get("architecture") != ARCHITECTURE:
            raise UnsupportedArchitectureError(
                f"config.json names architecture {raw.get('architecture')!r}; this class reads {ARCHITECTURE!r}")
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json key 'layers' must be a list with at least one layer")
        checked: List[Dict] = [_check_layer(i, layer) for i, layer in enumerate(layers)]
        values = dict(vocab=_int("", raw, "vocab"), width=_int("", raw, "width"), streams=_int("", raw, "streams"),
                      eps=_num("norm.", _table("", raw, "norm"), "eps"),
                      embedding_scale=_num("embedding.", _table("", raw, "embedding"), "scale", positive=False),
                      residual_mult=_num("", raw, "residual_mult", positive=False),
                      logit_scale=_num("", raw, "logit_scale", positive=False), layers=tuple(checked))
        if raw.get("max_positions") is not None:
            values["max_positions"] = _int("", raw, "max_positions")
        eos = raw.get("eos_token_id")
        if eos is not None:
            ids = list(eos) if isinstance(eos, (list, tuple)) else [eos]
            for t in ids:
                if isinstance(t, bool) or not isinstance(t, int) or not 0 <= t < values["vocab"]:
                    raise ConfigError(f"config.json key 'eos_token_id' must name token ids below vocab, found {eos!r}")
            values["eos_token_id"] = tuple(ids)
        return cls(**values)

    def to_dict(self) -> Dict:
        d = {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "streams": self.streams, "norm": {"eps": self.eps},
             "embedding": {"scale": self.embedding_scale}, "residual_mult": self.residual_mult, "logit_scale": self.logit_scale,
             "layers": copy.deepcopy(list(self.layers))}
        if self.max_positions is not None:
            d["max_positions"] = self.max_positions
        if self.eos_token_id is not None:
            d["eos_token_id"] = list(self.eos_token_id)
        return d

    def with_shapes(self, shapes: Dict[str, Tuple[int, ...]]) -> "NazulornConfig":
        """The configuration with what only the checkpoint's tensor shapes say filled in: the inner width of every decay's two
        small matrices (``l<i>.mix.a1`` is ``[rank, width]``)."""
        layers = []
        for i, layer in enumerate(self.layers):
            layer = copy.deepcopy(layer)
            if layer["type"] == "gla" and layer["mixer"].get("decay_rank") is None:
                shape = shapes.get(f"l{i}.mix.a1")
                if shape is not None and len(shape) == 2:
                    layer["mixer"]["decay_rank"] = int(shape[0])
            layers.append(layer)
        return replace(self, layers=tuple(layers))

    def _mixer(self, layer: Dict):
        m = layer["mixer"]
        if layer["type"] == "gla":
            return GatedLinearAttentionSpec(hidden=self.width, n_heads=m["heads"], head_dim=m["dim"], v_head_dim=m["vdim"],
                                            decay_rank=m.get("decay_rank") or DEFAULT_DECAY_RANK, tau=float(m["tau"]), eps=self.eps)
        position = None
        if m.get("rot") is not None:
            rot, sc = m["rot"], m["rot"].get("scaling")
            stretch = None if sc is None else RopeStretch(*(float(sc[k]) for k in ("factor", "original", "fast", "slow")))
            position = RopeSpec(head_dim=m["dim"], rot_dim=rot["dims"], theta=float(rot["base"]), stretch=stretch)
        return DifferentialAttentionSpec(hidden=self.width, n_heads=m["heads"], n_kv_heads=m["kv_heads"], head_dim=m["dim"],
                                         v_head_dim=m["vdim"], scale=float(m["scale"]), diff=float(m["diff"]), eps=self.eps,
                                         window=(m.get("mask") or {}).get("size"), position=position)

    def _feed_forward(self, mlp: Optional[Dict]):
        if mlp is None:
            return None
        r, e, shared = mlp["router"], mlp["expert"], mlp.get("shared")

        def limit(d: Optional[Dict]) -> Optional[float]:
            return None if d is None or d.get("limit") is None else float(d["limit"])
        scale = r.get("scale")
        return RoutedExpertsSpec(hidden=self.width, n_experts=r["experts"], identity=r.get("identity") or 0, top=r["top"],
                                 intermediate=e["ff"], activation=EXPERT_ACTIVATION, limit=limit(e), up_offset=EXPERT_UP_OFFSET,
                                 sum_eps=EXPERT_SUM_EPS, weighting="softmax_all", correction=True,
                                 weight_scale=1.0 if scale is None else float(scale),
                                 shared_intermediate=None if shared is None else shared["ff"], shared_limit=limit(shared))

    def to_model_spec(self) -> ModelSpec:
        def norm() -> NormSpec:
            return NormSpec(size=self.width, eps=self.eps)
        blocks = []
        for layer in self.layers:
            ffn = self._feed_forward(layer.get("mlp"))
            blocks.append(BlockSpec(mixer=self._mixer(layer), ffn=ffn, mixer_norm=norm(), ffn_norm=None if ffn is None else norm(),
                                    arrangement="linked_streams", streams=self.streams, branch_scale=self.residual_mult))
        spec = ModelSpec(architecture=ARCHITECTURE, vocab=self.vocab, hidden=self.width, layers=tuple(blocks),
                         schedule=default_schedule(len(blocks)), final_norm=norm(), tie_lm_head=False,
                         max_positions=self.max_positions or UNBOUNDED_POSITIONS, embed_scale=self.embedding_scale,
                         eos_token_ids=self.eos_token_id or (), logit_scale=self.logit_scale)
        spec.validate()
        return spec


def checkpoint_names(spec: ModelSpec) -> Dict[str, str]:
    """Internal parameter name -> tensor name in the checkpoint: ``embed``, ``head``, ``final.norm``, ``l<i>.norm1|norm2``,
    ``l<i>.hc1|hc2.in|out|mix``, ``l<i>.mix.q|k|v|o|lq1|lk1|lq2|lk2`` (attention) or ``l<i>.mix.q|k|v|g|o|norm|a1|a2|a2.b``,
    ``l<i>.mlp.router|correction``, ``l<i>.mlp.e<j>.gate|up|down`` and ``l<i>.mlp.shared.gate|up|down``."""
    names = {"embed.weight": "embed", "lm_head.weight": "head", "final_norm.weight": "final.norm"}
    for i, block in enumerate(spec.layers):
        src, dst = f"l{i}.", f"layers.{i}."
        sublayers = [("mixer", "1")] + ([("ffn", "2")] if block.ffn is not None else [])
        for sublayer, q in sublayers:
            names[dst + sublayer + "_norm.weight"] = src + "norm" + q
            for p in ("in", "out", "mix"):
                names[dst + f"{sublayer}_link.{p}"] = src + f"hc{q}.{p}"
        gla = block.mixer.kind == "gated_linear_attention"
        for p in ("q", "k", "v", "o") + (("g",) if gla else ()):
            names[dst + f"mixer.{p}_proj.weight"] = src + f"mix.{p}"
        if gla:
            for internal, stored in (("norm.weight", "norm"), ("a1.weight", "a1"), ("a2.weight", "a2"), ("a2.bias", "a2.b")):
                names[dst + "mixer." + internal] = src + "mix." + stored
        else:
            for p in ("lq1", "lk1", "lq2", "lk2"):
                names[dst + "mixer." + p] = src + "mix." + p
        if block.ffn is None:
            continue
        names[dst + "ffn.router.weight"], names[dst + "ffn.correction"] = src + "mlp.router", src + "mlp.correction"
        for p in ("gate", "up", "down"):
            for e in range(block.ffn.n_experts):
                names[dst + f"ffn.experts.{e}.{p}_proj.weight"] = src + f"mlp.e{e}.{p}"
            if block.ffn.shared_intermediate is not None:
                names[dst + f"ffn.shared.{p}_proj.weight"] = src + f"mlp.shared.{p}"
    return names


def unused_tensors(spec: ModelSpec) -> Tuple[str, ...]:
    """Tensors a checkpoint may hold that the model does not read: the second norm and links of a layer without a feed-forward."""
    out = []
    for i, block in enumerate(spec.layers):
        if block.ffn is None:
            out += [f"l{i}.norm2", f"l{i}.hc2.in", f"l{i}.hc2.out", f"l{i}.hc2.mix"]
    return tuple(out)
