"""Sonulorn configuration: a list of layers whose mixer and feed-forward read the same norm of the stream side by side, each
with one of three mixers, and a run of layers that is passed through several times with the same weights.

config.json keys: ``architecture`` ("Sonulorn"), ``vocab``, ``width``, ``norm`` {eps}, ``embedding`` {scale}, ``loop`` {start,
stop, times} and ``layers``: a list of ``{"type", "mixer", "mlp"}``.  ``type`` names the mixer:

  ``attention``  ``mixer`` = {heads, kv_heads, dim, vdim, scale, rot: {dims, base}, mask: {size}}
  ``parallel``   ``mixer`` = {left: {heads, kv_heads, dim, vdim, scale, conv, rot: {dims, base}},
                              right: {heads, kv_heads, dim, vdim, conv}, left_scale, right_scale}
  ``lightning``  ``mixer`` = {heads, dim, vdim, decay: [one a head]}

``kv_heads`` (as many as ``heads``), ``vdim`` (``dim``), ``scale`` (one over the root of a key's size), ``rot`` (no rotation),
``mask`` (every earlier key is seen), ``left.conv`` (no convolution), ``left_scale`` and ``right_scale`` (1), ``embedding.scale``
(1) and ``loop`` (every layer runs once) may be absent.  ``mlp`` is null or {kind: "dense", ff, limit}.  ``max_positions``
(optional) bounds the rotary tables and a request's length.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, field
from typing import Any, Dict, Mapping, Optional, Tuple, Union

from .base import ConfigError, FieldReader

DEFAULT_MAX_POSITIONS = 32768


class _Reader(FieldReader):
    """A field reader whose errors carry the path of the object it reads."""

    def __init__(self, raw: Mapping[str, Any], where: str = ""):
        super().__init__(raw)
        self.where = where

    def _located(self, read, *args):
        try:
            return read(*args)
        except ConfigError as error:
            raise ConfigError(self.where + error.field, str(error).split(": ", 2)[-1]) from None

    def size(self, key: str, *default) -> int:
        return self._located(self.positive_int, key, *default)

    def real(self, key: str, *default) -> float:
        return self._located(self.positive_float, key, *default)

    def number(self, key: str, default: Optional[float] = None) -> float:
        """A finite number of either sign."""
        value = self.optional(key)
        if value is None and default is not None:
            return default
        if isinstance(value, bool) or not isinstance(value, (int, float)) or not math.isfinite(float(value)):
            raise ConfigError(self.where + key, f"expected a finite number, found {value!r}")
        return float(value)

    def inner(self, key: str, optional: bool = False) -> Optional["_Reader"]:
        value = self.optional(key)
        if value is None and optional:
            return None
        if not isinstance(value, dict):
            raise ConfigError(self.where + key, f"expected an object, found {value!r}")
        return _Reader(value, f"{self.where}{key}.")

    def grouped_heads(self) -> Tuple[int, int]:
        heads = self.size("heads")
        kv_heads = self.size("kv_heads", heads)
        if heads % kv_heads:
            raise ConfigError(self.where + "kv_heads", f"{heads} heads cannot be grouped over {kv_heads} key heads")
        return heads, kv_heads


@dataclass(frozen=True)
class SinkAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_dims: Optional[int]       # None: no rotation
    rot_base: Optional[float]
    chunk: Optional[int]          # None: every earlier key is seen
    taps: Optional[int] = None    # None: no convolutions behind the projections

    @classmethod
    def read(cls, r: _Reader, mask: bool, conv: bool) -> "SinkAttentionConfig":
        heads, kv_heads = r.grouped_heads()
        dim = r.size("dim")
        rot, dims, base = r.inner("rot", optional=True), None, None
        if rot is not None:
            dims, base = rot.size("dims"), rot.real("base")
            if dims % 2 or dims > dim:
                raise ConfigError(rot.where + "dims", f"must be even and at most the head's {dim}, found {dims}")
        masked = r.inner("mask", optional=True) if mask else None
        return cls(heads, kv_heads, dim, r.size("vdim", dim), r.real("scale", dim ** -0.5), dims, base,
                   masked.size("size") if masked is not None else None, r.size("conv", None) if conv else None)

    def to_dict(self) -> dict:
        out: Dict[str, Any] = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.rot_dims is not None:
            out["rot"] = {"dims": self.rot_dims, "base": self.rot_base}
        if self.chunk is not None:
            out["mask"] = {"size": self.chunk}
        if self.taps is not None:
            out["conv"] = self.taps
        return out


@dataclass(frozen=True)
class HeadDeltaConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int

    def to_dict(self) -> dict:
        return {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "conv": self.taps}


@dataclass(frozen=True)
class ParallelConfig:
    left: SinkAttentionConfig
    right: HeadDeltaConfig
    left_scale: float
    right_scale: float

    def to_dict(self) -> dict:
        return {"left": self.left.to_dict(), "right": self.right.to_dict(), "left_scale": self.left_scale, "right_scale": self.right_scale}


@dataclass(frozen=True)
class LightningConfig:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]

    def to_dict(self) -> dict:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "decay": list(self.decay)}


@dataclass(frozen=True)
class DenseConfig:
    ff: int
    limit: float


@dataclass(frozen=True)
class LoopConfig:
    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class SonulornLayer:
    type: str
    mixer: Union[SinkAttentionConfig, ParallelConfig, LightningConfig]
    mlp: Optional[DenseConfig]        # None: the layer has no feed-forward


def _attention(r: _Reader) -> SinkAttentionConfig:
    return SinkAttentionConfig.read(r, mask=True, conv=False)


def _parallel(r: _Reader) -> ParallelConfig:
    left, right = r.inner("left"), r.inner("right")
    memory = HeadDeltaConfig(*right.grouped_heads(), right.size("dim"), right.size("vdim", right.size("dim")), right.size("conv"))
    return ParallelConfig(SinkAttentionConfig.read(left, mask=False, conv=True), memory, r.number("left_scale", 1.0),
                          r.number("right_scale", 1.0))


def _lightning(r: _Reader) -> LightningConfig:
    heads, dim = r.size("heads"), r.size("dim")
    decay = r.optional("decay")
    if not isinstance(decay, list) or len(decay) != heads or not all(
            isinstance(d, (int, float)) and not isinstance(d, bool) and 0.0 <= d <= 1.0 for d in decay):
        raise ConfigError(r.where + "decay", f"expected {heads} numbers in [0, 1], found {decay!r}")
    return LightningConfig(heads, dim, r.size("vdim", dim), tuple(float(d) for d in decay))


_MIXERS = {"attention": _attention, "parallel": _parallel, "lightning": _lightning}


def _layer(entry: Any, where: str) -> SonulornLayer:
    if not isinstance(entry, dict):
        raise ConfigError(where[:-1], f"expected an object, found {entry!r}")
    r = _Reader(entry, where)
    kind = r.optional("type")
    if kind not in _MIXERS:
        raise ConfigError(where + "type", f"unknown layer type {kind!r}; known: {', '.join(sorted(_MIXERS))}")
    mixer = _MIXERS[kind](r.inner("mixer"))
    f = r.inner("mlp", optional=True)
    if f is None:
        return SonulornLayer(kind, mixer, None)
    if f.optional("kind") != "dense":
        raise ConfigError(f.where + "kind", f"expected \"dense\", found {f.optional('kind')!r}")
    return SonulornLayer(kind, mixer, DenseConfig(f.size("ff"), f.real("limit")))


def _loop(r: Optional[_Reader], layers: int) -> Optional[LoopConfig]:
    if r is None:
        return None
    bounds = []
    for key in ("start", "stop"):
        value = r.optional(key)
        if isinstance(value, bool) or not isinstance(value, int) or not 0 <= value <= layers:
            raise ConfigError(r.where + key, f"expected a number of layers from 0 to {layers}, found {value!r}")
        bounds.append(value)
    if bounds[0] >= bounds[1]:
        raise ConfigError(r.where + "stop", f"the loop holds no layer: {bounds[0]} .. {bounds[1]}")
    return LoopConfig(*bounds, r.size("times"))


@dataclass(frozen=True)
class SonulornConfig:
    architecture: str
    vocab: int
    width: int
    eps: float
    embedding_scale: float
    layers: Tuple[SonulornLayer, ...]
    loop: Optional[LoopConfig]        # None: every layer runs once
    max_positions: int = DEFAULT_MAX_POSITIONS
    raw: Dict[str, Any] = field(default_factory=dict, compare=False, repr=False)

    ARCHITECTURE = "Sonulorn"

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any]) -> "SonulornConfig":
        r = _Reader(raw)
        listed = r.optional("layers")
        if not isinstance(listed, list) or not listed:
            raise ConfigError("layers", "expected a list of layers")
        layers = tuple(_layer(entry, f"layers[{i}].") for i, entry in enumerate(listed))
        embedding = r.inner("embedding", optional=True)
        return cls(cls.ARCHITECTURE, r.size("vocab"), r.size("width"), r.inner("norm").real("eps"),
                   embedding.number("scale", 1.0) if embedding is not None else 1.0, layers,
                   _loop(r.inner("loop", optional=True), len(layers)), r.size("max_positions", DEFAULT_MAX_POSITIONS),
                   {k: v for k, v in raw.items() if k != "torch_dtype"})

    def to_dict(self) -> dict:
        """The config.json that reads back as this configuration."""
        out: Dict[str, Any] = {
            "architecture": self.ARCHITECTURE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
            "embedding": {"scale": self.embedding_scale},
            "layers": [{"type": layer.type, "mixer": layer.mixer.to_dict(),
                        "mlp": None if layer.mlp is None else {"kind": "dense", "ff": layer.mlp.ff, "limit": layer.mlp.limit}}
                       for layer in self.layers]}
        if self.loop is not None:
            out["loop"] = {"start": self.loop.start, "stop": self.loop.stop, "times": self.loop.times}
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
