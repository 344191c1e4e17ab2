"""Typed configuration of the Kakalorn decoder, read from config.json.

A Kakalorn layer has a norm before and one after each sublayer, ``x += norm1b(mixer(norm1(x)))`` and
``x += norm2b(ff(norm2(x)))``, all of them root-mean-square norms with a plain gain.  What a mixer reads is first
replaced by itself plus a short causal convolution over it.  A layer's mixer is

* a **windowed attention** (``type: attention``): grouped heads, biased q and k whose per-head norm and rotation come
  behind the projection, values that are the projected keys, a window beside which the first positions stay visible, and
  a learned sink per head;
* a **recurrence** (``type: hgrn2``): linear attention whose forget gate, held above a learned lower bound, also decides
  what is written; or
* a **latent attention** (``type: latent_attention``): queries through a latent, keys and values expanded from one latent
  row per position plus a rotated part that the heads share (pairs of neighbours, frequencies that may be slowed down), a
  gate per head.  A layer may run on the rows that an earlier latent layer keeps (``kv_from``).

The feed-forward is ``W_down max(W_up h, 0)^2`` or absent; the output matrix is its own.  config.json gives every size
layer by layer:

* ``architecture``: ``"Kakalorn"``; ``vocab``, ``width``; ``norm.eps``; ``canon.taps``; ``max_positions`` or absent;
* ``layers[i]``: ``type``; ``mixer``: for ``attention`` ``heads``, ``kv_heads``, ``dim``, ``vdim`` (equal to ``dim``),
  ``scale``, ``mask`` (``size``, ``keep_first``) and ``rot`` (``base``, ``dims``); for ``hgrn2`` ``heads``, ``dim``, ``vdim``;
  for ``latent_attention`` ``heads``, ``dim``, ``rot_dim``, ``vdim``, ``q_rank``, ``kv_rank``, ``scale``, ``rot`` (``base``,
  ``dims`` equal to ``rot_dim``, ``scaling`` with ``factor``, ``original``, ``fast``, ``slow``, or absent) and ``kv_from`` or
  absent; ``mlp``: null or ``{"kind": "dense", "ff": n}``.

Constants the design fixes live here: the feed-forward's activation, the pairings of the rotations.
"""
from __future__ import annotations

import copy
import math
from dataclasses import dataclass
from typing import Dict, List, Optional, Tuple

from ..errors import ConfigError, UnsupportedArchitectureError
from .spec import (AttentionSpec, BlockSpec, Hgrn2Spec, LatentAttentionSpec, MlpSpec, ModelSpec, NormSpec, RopeSpec, RopeStretch,
                   ScheduleEntry)

ARCHITECTURE = "Kakalorn"
ACTIVATION = "relu2"
ATTENTION_PAIRING, LATENT_PAIRING = "halves", "neighbours"
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


def _num(where: str, d: Dict, key: str) -> float:
    if key not in d:
        raise ConfigError(f"config.json lacks {where}{key!r}")
    v = d[key]
    if isinstance(v, bool) or not isinstance(v, (int, float)) or not math.isfinite(v) or v <= 0:
        raise ConfigError(f"config.json {where}{key!r} must be a positive number, found {v!r}")
    return float(v)


def _check_rot(where: str, m: Dict, most: int, whole: bool) -> None:
    rot = _table(where, m, "rot")
    base, dims = _num(where + "rot.", rot, "base"), _int(where + "rot.", rot, "dims")
    if dims % 2 != 0 or dims > most or (whole and dims != most):
        raise ConfigError(f"config.json {where}rot.dims must be even and {'equal to' if whole else 'at most'} {most}, found {dims}")
    if rot.get("scaling") is not None:
        sc = _table(where + "rot.", rot, "scaling")
        for key in ("factor", "original", "fast", "slow"):
            _num(where + "rot.scaling.", sc, key)
        if base <= 1.0:
            raise ConfigError(f"config.json {where}rot.base must be above 1 where its frequencies are scaled, found {base}")


def _check_layer(i: int, layer, before: List[Dict]) -> Dict:
    where = f"layers[{i}]."
    kind = layer.get("type") if isinstance(layer, dict) else None
    if kind not in ("attention", "hgrn2", "latent_attention"):
        raise ConfigError(f"config.json {where}type is {kind!r}; known: attention, hgrn2, latent_attention")
    m, w = _table(where, layer, "mixer"), where + "mixer."
    for key in ("heads", "dim", "vdim"):
        _int(w, m, key)
    if kind == "attention":
        _int(w, m, "kv_heads")
        _num(w, m, "scale")
        if m["heads"] % m["kv_heads"] != 0:
            raise ConfigError(f"config.json {w[:-1]}: {m['heads']} heads are not a multiple of {m['kv_heads']} kv_heads")
        if m["vdim"] != m["dim"]:
            raise ConfigError(f"config.json {w}vdim must equal dim ({m['dim']}): the values are the keys, found {m['vdim']}")
        mask = _table(w, m, "mask")
        _int(w + "mask.", mask, "size")
        _int(w + "mask.", mask, "keep_first", least=0)
        _check_rot(w, m, m["dim"], whole=False)
    elif kind == "latent_attention":
        for key in ("rot_dim", "q_rank", "kv_rank"):
            _int(w, m, key)
        _num(w, m, "scale")
        _check_rot(w, m, m["rot_dim"], whole=True)
        src = m.get("kv_from")
        if src is not None:
            if isinstance(src, bool) or not isinstance(src, int) or not 0 <= src < i or before[src]["type"] != "latent_attention" \
                    or before[src]["mixer"].get("kv_from") is not None:
                raise ConfigError(f"config.json {w}kv_from must name an earlier latent attention layer with rows of its own, found {src!r}")
            other = before[src]["mixer"]
            for key in ("kv_rank", "rot_dim", "rot"):
                if other.get(key) != m.get(key):
                    raise ConfigError(f"config.json {w}{key} differs from layer {src}, whose rows the layer reads")
    mlp = layer.get("mlp")
    if mlp is not None:
        if not isinstance(mlp, dict) or mlp.get("kind") != "dense":
            raise ConfigError(f"config.json {where}mlp must be null or of kind 'dense', found {mlp!r}")
        _int(where + "mlp.", mlp, "ff")
    return copy.deepcopy(layer)


@dataclass(frozen=True)
class KakalornConfig:
    vocab: int
    width: int
    eps: float
    taps: int                              # of the convolution on every mixer's input
    layers: Tuple[Dict, ...]               # as config.json has them, validated
    max_positions: Optional[int] = None
    eos_token_id: Optional[Tuple[int, ...]] = None

    @classmethod
    def from_dict(cls, raw: Dict) -> "KakalornConfig":
        if raw.get("architecture") != ARCHITECTURE:
            raise UnsupportedArchitectureError(
                f"config.json names architecture {raw.get('architecture')!r}; this class reads {ARCHITECTURE!r}")
        vocab, width = _int("", raw, "vocab"), _int("", raw, "width")
        eps = _num("norm.", _table("", raw, "norm"), "eps")
        taps = _int("canon.", _table("", raw, "canon"), "taps")
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json key 'layers' must be a list with at least one layer")
        checked: List[Dict] = []
        for i, layer in enumerate(layers):
            checked.append(_check_layer(i, layer, checked))
        values = dict(vocab=vocab, width=width, eps=eps, taps=taps, layers=tuple(checked))
        if raw.get("max_positions") is not None:
            values["max_positions"] = _int("", raw, "max_positions")
        eos = raw.get("eos_token_id")
        if eos is not None:
            ids = list(eos) if isinstance(eos, (list, tuple)) else [eos]
            for t in ids:
                if isinstance(t, bool) or not isinstance(t, int) or not 0 <= t < vocab:
                    raise ConfigError(f"config.json key 'eos_token_id' must name token ids below vocab, found {eos!r}")
            values["eos_token_id"] = tuple(ids)
        return cls(**values)

    def to_dict(self) -> Dict:
        d = {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
             "canon": {"taps": self.taps}, "layers": copy.deepcopy(list(self.layers))}
        if self.max_positions is not None:
            d["max_positions"] = self.max_positions
        if self.eos_token_id is not None:
            d["eos_token_id"] = list(self.eos_token_id)
        return d

    def schedule(self) -> Tuple[ScheduleEntry, ...]:
        """Every layer once, in order; a layer with ``kv_from`` reads that layer's cache line."""
        return tuple(ScheduleEntry(layer=i, reads_cache_of=layer["mixer"].get("kv_from")) for i, layer in enumerate(self.layers))

    def _mixer(self, layer: Dict):
        m = layer["mixer"]
        if layer["type"] == "hgrn2":
            return Hgrn2Spec(hidden=self.width, n_heads=m["heads"], head_dim=m["dim"], v_head_dim=m["vdim"], eps=self.eps)
        rot = m["rot"]
        if layer["type"] == "attention":
            sc = rot.get("scaling")
            position = RopeSpec(head_dim=m["dim"], rot_dim=rot["dims"], theta=float(rot["base"]), pairing=ATTENTION_PAIRING,
                                stretch=None if sc is None else _stretch(sc))
            return AttentionSpec(hidden=self.width, n_heads=m["heads"], n_kv_heads=m["kv_heads"], head_dim=m["dim"], scale=float(m["scale"]),
                                 window=m["mask"]["size"], keep_first=m["mask"]["keep_first"],
                                 qk_norm=NormSpec(size=m["dim"], eps=self.eps), position=position, bias=True, o_bias=False,
                                 sink=True, sink_learned=True, values_are_keys=True)
        sc = rot.get("scaling")
        return LatentAttentionSpec(hidden=self.width, n_heads=m["heads"], head_dim=m["dim"], rot_dim=m["rot_dim"], v_head_dim=m["vdim"],
                                   q_rank=m["q_rank"], kv_rank=m["kv_rank"], scale=float(m["scale"]),
                                   q_norm=NormSpec(size=m["q_rank"], eps=self.eps), kv_norm=NormSpec(size=m["kv_rank"], eps=self.eps),
                                   position=RopeSpec(head_dim=m["rot_dim"], rot_dim=rot["dims"], theta=float(rot["base"]),
                                                     pairing=LATENT_PAIRING, stretch=None if sc is None else _stretch(sc)),
                                   gate=True, gate_per_head=True, own_rows=m.get("kv_from") is None)

    def to_model_spec(self) -> ModelSpec:
        def norm() -> NormSpec:
            return NormSpec(size=self.width, eps=self.eps)
        blocks = []
        for layer in self.layers:
            mlp = layer.get("mlp")
            ffn = None if mlp is None else MlpSpec(hidden=self.width, intermediate=mlp["ff"], activation=ACTIVATION)
            blocks.append(BlockSpec(mixer=self._mixer(layer), ffn=ffn, mixer_norm=norm(), ffn_norm=None if ffn is None else norm(),
                                    arrangement="sandwich_norm", mixer_out_norm=norm(), ffn_out_norm=None if ffn is None else norm(),
                                    input_conv=self.taps))
        spec = ModelSpec(architecture=ARCHITECTURE, vocab=self.vocab, hidden=self.width, layers=tuple(blocks),
                         schedule=self.schedule(), final_norm=norm(), tie_lm_head=False,
                         max_positions=self.max_positions or UNBOUNDED_POSITIONS, eos_token_ids=self.eos_token_id or ())
        spec.validate()
        return spec


def _stretch(sc: Dict) -> RopeStretch:
    return RopeStretch(factor=float(sc["factor"]), original=float(sc["original"]), fast=float(sc["fast"]), slow=float(sc["slow"]))


def checkpoint_names(spec: ModelSpec) -> Dict[str, str]:
    """Internal parameter name -> tensor name in the checkpoint: ``embed``, ``head``, ``final.norm``,
    ``l<i>.norm1|norm1b|norm2|norm2b``, ``l<i>.canon1``, ``l<i>.mix.q|k|o``, ``.q.b|k.b``, ``.q.norm|k.norm``, ``.sink``
    (attention), ``l<i>.mix.q|f|v|o``, ``.f.b``, ``.lower``, ``.norm`` (the recurrence), ``l<i>.mix.dq|uq|dkv|uk|uv|g|o``,
    ``.dq.norm|dkv.norm`` (latent attention; without ``dkv`` where the rows are another layer's), ``l<i>.mlp.up|down``."""
    names = {"embed.weight": "embed", "final_norm.weight": "final.norm", "lm_head.weight": "head"}
    for i, block in enumerate(spec.layers):
        src, dst = f"l{i}.", f"layers.{i}."
        names[dst + "mixer_norm.weight"], names[dst + "mixer_out_norm.weight"] = src + "norm1", src + "norm1b"
        names[dst + "input_conv.weight"] = src + "canon1"
        mix, own = src + "mix.", dst + "mixer."
        if block.mixer.kind == "attention":
            for p in ("q", "k"):
                names[own + f"{p}_proj.weight"], names[own + f"{p}_proj.bias"] = mix + p, mix + p + ".b"
                names[own + f"{p}_norm.weight"] = mix + p + ".norm"
            names[own + "sink"], names[own + "o_proj.weight"] = mix + "sink", mix + "o"
        elif block.mixer.kind == "hgrn2":
            for p in ("q", "f", "v", "o"):
                names[own + f"{p}_proj.weight"] = mix + p
            names[own + "f_proj.bias"], names[own + "lower"], names[own + "norm.weight"] = mix + "f.b", mix + "lower", mix + "norm"
        else:
            for p in ("dq", "uq", "uk", "uv", "g") + (("dkv",) if block.mixer.own_rows else ()):
                names[own + f"{p}.weight"] = mix + p
            names[own + "dq_norm.weight"], names[own + "o_proj.weight"] = mix + "dq.norm", mix + "o"
            if block.mixer.own_rows:
                names[own + "dkv_norm.weight"] = mix + "dkv.norm"
        if block.ffn is None:
            continue
        names[dst + "ffn_norm.weight"], names[dst + "ffn_out_norm.weight"] = src + "norm2", src + "norm2b"
        for p in ("up", "down"):
            names[dst + f"ffn.{p}_proj.weight"] = src + f"mlp.{p}"
    return names


def unused_tensors(spec: ModelSpec) -> Tuple[str, ...]:
    """Tensors a checkpoint may hold that the model does not read: the second norms of a layer without a feed-forward."""
    return tuple(f"l{i}.{n}" for i, block in enumerate(spec.layers) if block.ffn is None for n in ("norm2", "norm2b"))
