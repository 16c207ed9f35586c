"""Reverax configuration: a list of layers whose mixer and feed-forward read the same stream side by side, each with one of
two mixers (softmax attention whose heads' scores are mixed, or softmax attention with turned values beside a matrix
memory with token-made decays) and a dense or routed feed-forward (or none).

config.json keys: ``architecture`` ("Reverax"), ``vocab``, ``width``, ``norm`` {eps, groups}, ``logit_scale`` and
``layers``: a list of ``{"type", "mixer", "mlp", "weights_of"}``.  ``type`` names the mixer:

  ``attention``  ``mixer`` = {heads, kv_heads, dim, vdim, scale, rot: {dims, base}}
  ``parallel``   ``mixer`` = {left: {heads, kv_heads, dim, vdim, scale, softcap, rot: {dims, base}, mask: {size}},
                              right: {heads, dim}, left_scale, right_scale}

``mask`` (every earlier key is seen), ``softcap``, ``kv_heads`` (as many as ``heads``), ``vdim`` (``dim``), ``scale`` (one over
the root of a key's size), ``norm.groups`` and ``logit_scale`` (1) may be absent.  ``mlp`` is null, {kind: "dense", ff} or
{kind: "moe", expert: {ff}, router: {experts, top}}.  ``weights_of``: the layer has no tensors of its own and takes those of
the layer named, with a cache of its own; the rest of its entry, where given, equals that layer's.  The rank of the memory's
low-rank decay is not in config.json; it is read from the tensors' shapes when the weights are bound (``with_shapes``), and a
folder written from a configuration notes it as ``right.decay_rank``.  ``max_positions`` (optional) bounds the rotary
tables and a request's length.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, replace
from typing import Any, Dict, List, Mapping, Optional, Tuple, Union

from .base import ConfigError, FieldReader

DEFAULT_MAX_POSITIONS = 32768


def _sub(raw: Mapping[str, Any], key: str, where: str, optional: bool = False) -> Optional[FieldReader]:
    value = raw.get(key)
    if value is None and optional:
        return None
    if not isinstance(value, dict):
        raise ConfigError(f"{where}{key}", f"expected an object, found {value!r}")
    return FieldReader(value)


def _relabel(error: ConfigError, where: str) -> ConfigError:
    if error.field.startswith(where) or error.field.startswith("layers["):
        return error
    return ConfigError(where + error.field, str(error).split(": ", 2)[-1])


def _number(reader: FieldReader, key: str) -> float:
    """A finite number of either sign (a branch's weight)."""
    value = reader.optional(key)
    if isinstance(value, bool) or not isinstance(value, (int, float)) or not math.isfinite(float(value)):
        raise ConfigError(key, f"expected a finite number, found {value!r}")
    return float(value)


@dataclass(frozen=True)
class TalkingAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_dims: int
    rot_base: float


@dataclass(frozen=True)
class TurnedAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_dims: int
    rot_base: float
    softcap: Optional[float]      # None: scores are taken as they are
    window: Optional[int]         # None: every earlier key is seen


@dataclass(frozen=True)
class TimeMixConfig:
    heads: int
    dim: int
    decay_rank: Optional[int] = None      # from the tensors' shapes


@dataclass(frozen=True)
class ParallelConfig:
    left: TurnedAttentionConfig
    right: TimeMixConfig
    left_scale: float
    right_scale: float


@dataclass(frozen=True)
class DenseConfig:
    ff: int


@dataclass(frozen=True)
class MixtureConfig:
    experts: int
    top: int
    expert_ff: int


@dataclass(frozen=True)
class LayerConfig:
    kind: str                     # "attention" or "parallel"
    mixer: Union[TalkingAttentionConfig, ParallelConfig]
    mlp: Union[None, DenseConfig, MixtureConfig]
    weights_of: Optional[int] = None


def _heads(m: FieldReader, where: str) -> Tuple[int, int, int, int, float, int, float]:
    """(heads, kv_heads, dim, vdim, scale, rotated elements, base of the rotation) of an attention."""
    heads, dim = m.positive_int("heads"), m.positive_int("dim")
    kv_heads, vdim = m.positive_int("kv_heads", heads), m.positive_int("vdim", dim)
    scale = m.positive_float("scale", dim ** -0.5)
    rot = _sub(m.raw, "rot", where)
    try:
        dims, base = rot.positive_int("dims"), rot.positive_float("base")
    except ConfigError as error:
        raise _relabel(error, where + "rot.") from None
    if dims % 2 or dims > dim:
        raise ConfigError(where + "rot.dims", f"must be even and at most {dim}, found {dims}")
    if base <= 1.0:
        raise ConfigError(where + "rot.base", f"must be above 1, found {base}")
    if heads % kv_heads:
        raise ConfigError(where + "kv_heads", f"{heads} query heads cannot be grouped over {kv_heads} key/value heads")
    return heads, kv_heads, dim, vdim, scale, dims, base


def _talking(raw: Mapping[str, Any], where: str) -> TalkingAttentionConfig:
    m, w = _sub(raw, "mixer", where), where + "mixer."
    try:
        return TalkingAttentionConfig(*_heads(m, w))
    except ConfigError as error:
        raise _relabel(error, w) from None


def _parallel(raw: Mapping[str, Any], where: str) -> ParallelConfig:
    m, w = _sub(raw, "mixer", where), where + "mixer."
    left, right = _sub(m.raw, "left", w), _sub(m.raw, "right", w)
    try:
        shape = _heads(left, w + "left.")
        cap = left.positive_float("softcap") if left.has("softcap") else None
        mask = _sub(left.raw, "mask", w + "left.", optional=True)
        try:
            window = mask.positive_int("size") if mask is not None else None
        except ConfigError as error:
            raise _relabel(error, w + "left.mask.") from None
    except ConfigError as error:
        raise _relabel(error, w + "left.") from None
    if shape[3] % 2:
        raise ConfigError(w + "left.vdim", f"values that turn in pairs have an even size, found {shape[3]}")
    try:
        memory = TimeMixConfig(right.positive_int("heads"), right.positive_int("dim"), right.positive_int("decay_rank", None))
    except ConfigError as error:
        raise _relabel(error, w + "right.") from None
    try:
        scales = _number(m, "left_scale"), _number(m, "right_scale")
    except ConfigError as error:
        raise _relabel(error, w) from None
    return ParallelConfig(TurnedAttentionConfig(*shape, cap, window), memory, *scales)


def _mlp(raw: Mapping[str, Any], where: str):
    if raw.get("mlp") is None:
        return None
    f, w = _sub(raw, "mlp", where), where + "mlp."
    kind = f.optional("kind")
    try:
        if kind == "dense":
            return DenseConfig(f.positive_int("ff"))
        if kind != "moe":
            raise ConfigError(w + "kind", f"expected \"dense\" or \"moe\", found {kind!r}")
        expert, router = _sub(f.raw, "expert", w), _sub(f.raw, "router", w)
        try:
            ff = expert.positive_int("ff")
        except ConfigError as error:
            raise _relabel(error, w + "expert.") from None
        try:
            experts, top = router.positive_int("experts"), router.positive_int("top")
        except ConfigError as error:
            raise _relabel(error, w + "router.") from None
    except ConfigError as error:
        raise _relabel(error, w) from None
    if top > experts:
        raise ConfigError(w + "router.top", f"{top} of {experts} experts cannot be chosen")
    return MixtureConfig(experts, top, ff)


_MIXERS = {"attention": _talking, "parallel": _parallel}


def _layers(listed: List[Any]) -> Tuple[LayerConfig, ...]:
    """The layers in order.  One that takes another's weights has that layer's mixer and feed-forward, and names the layer
    that owns the tensors (which may itself have been named through a third)."""
    def entry(i: int) -> Mapping[str, Any]:
        if not isinstance(listed[i], dict):
            raise ConfigError(f"layers[{i}]", f"expected an object, found {listed[i]!r}")
        return listed[i]

    def owner(i: int) -> int:
        seen = [i]
        while entry(seen[-1]).get("weights_of") is not None:
            j = entry(seen[-1])["weights_of"]
            if isinstance(j, bool) or not isinstance(j, int) or not 0 <= j < len(listed) or j in seen:
                raise ConfigError(f"layers[{i}].weights_of", f"must name another layer with tensors of its own, found {j!r}")
            seen.append(j)
        return seen[-1]

    def own(i: int) -> LayerConfig:
        where, kind = f"layers[{i}].", entry(i).get("type")
        if kind not in _MIXERS:
            raise ConfigError(where + "type", f"expected one of {', '.join(sorted(_MIXERS))}, found {kind!r}")
        return LayerConfig(kind, _MIXERS[kind](listed[i], where), _mlp(listed[i], where))

    found = {i: own(i) for i in range(len(listed)) if owner(i) == i}
    layers = []
    for i in range(len(listed)):
        j = owner(i)
        if j != i:
            for key in ("type", "mixer", "mlp"):
                if key in listed[i] and listed[i][key] != listed[j].get(key):
                    raise ConfigError(f"layers[{i}].{key}", f"a layer with the weights of layer {j} has that layer's {key}")
        layers.append(found[i] if j == i else replace(found[j], weights_of=j))
    return tuple(layers)


@dataclass(frozen=True)
class ReveraxConfig:
    vocab: int
    width: int
    eps: float
    norm_groups: int
    layers: Tuple[LayerConfig, ...]
    logit_scale: float = 1.0
    max_positions: int = DEFAULT_MAX_POSITIONS
    architecture: str = "Reverax"

    ARCHITECTURE = "Reverax"

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any]) -> "ReveraxConfig":
        top = FieldReader(raw)
        vocab, width = top.positive_int("vocab"), top.positive_int("width")
        norm = _sub(raw, "norm", "")
        try:
            eps, groups = norm.positive_float("eps"), norm.positive_int("groups", 1)
        except ConfigError as error:
            raise _relabel(error, "norm.") from None
        if width % groups:
            raise ConfigError("norm.groups", f"{width} elements cannot be normed in {groups} equal parts")
        listed = raw.get("layers")
        if not isinstance(listed, list) or not listed:
            raise ConfigError("layers", f"expected a list of layers, found {listed!r}")
        return cls(vocab, width, eps, groups, _layers(listed),
                   logit_scale=_number(top, "logit_scale") if top.has("logit_scale") else 1.0,
                   max_positions=top.positive_int("max_positions", DEFAULT_MAX_POSITIONS))

    def with_shapes(self, shapes: Mapping[str, tuple]) -> "ReveraxConfig":
        """The configuration with the sizes that only the tensors give: the ranks of the low-rank decays."""
        def known(i: int, layer: LayerConfig) -> LayerConfig:
            w1 = shapes.get(f"l{i if layer.weights_of is None else layer.weights_of}.mix.right.w1")
            if not isinstance(layer.mixer, ParallelConfig) or w1 is None or len(w1) != 2:
                return layer
            return replace(layer, mixer=replace(layer.mixer, right=replace(layer.mixer.right, decay_rank=int(w1[0]))))
        return replace(self, layers=tuple(known(i, layer) for i, layer in enumerate(self.layers)))

    def with_ranks(self, decay_rank: int) -> "ReveraxConfig":
        """The same for a model made from random weights: every memory's decay gets this rank."""
        return replace(self, layers=tuple(
            replace(layer, mixer=replace(layer.mixer, right=replace(layer.mixer.right, decay_rank=decay_rank)))
            if isinstance(layer.mixer, ParallelConfig) else layer for layer in self.layers))

    def to_dict(self) -> Dict[str, Any]:
        def attention(m) -> Dict[str, Any]:
            return {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "scale": m.scale,
                    "rot": {"dims": m.rot_dims, "base": m.rot_base}}

        layers = []
        for layer in self.layers:
            m = layer.mixer
            if isinstance(m, TalkingAttentionConfig):
                mixer: Dict[str, Any] = attention(m)
            else:
                left, right = attention(m.left), {"heads": m.right.heads, "dim": m.right.dim}
                if m.left.softcap is not None:
                    left["softcap"] = m.left.softcap
                if m.left.window is not None:
                    left["mask"] = {"size": m.left.window}
                if m.right.decay_rank is not None:
                    right["decay_rank"] = m.right.decay_rank
                mixer = {"left": left, "right": right, "left_scale": m.left_scale, "right_scale": m.right_scale}
            f = layer.mlp
            if f is None:
                mlp = None
            elif isinstance(f, DenseConfig):
                mlp = {"kind": "dense", "ff": f.ff}
            else:
                mlp = {"kind": "moe", "expert": {"ff": f.expert_ff}, "router": {"experts": f.experts, "top": f.top}}
            entry = {"type": layer.kind, "mixer": mixer, "mlp": mlp}
            if layer.weights_of is not None:
                entry["weights_of"] = layer.weights_of
            layers.append(entry)
        out: Dict[str, Any] = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
                               "norm": {"eps": self.eps, "groups": self.norm_groups}, "logit_scale": self.logit_scale,
                               "layers": layers}
        if self.max_positions != DEFAULT_MAX_POSITIONS:
            out["max_positions"] = self.max_positions
        return out

    # what the generic entry points ask a configuration for
    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def max_position_embeddings(self) -> int:
        return self.max_positions

    eos_token_id = None
