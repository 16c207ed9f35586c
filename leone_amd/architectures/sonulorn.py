"""Sonulorn: how its configuration becomes parts.

A small decoder-only design whose config.json lists its layers one by one.  A layer's mixer and feed-forward read one norm of
the stream and are added together (``parallel_prenorm`` block with one norm): x <- x + mixer(norm1(x)) + ff(norm1(x)).  Three
mixers:

* ``attention``: grouped-query softmax attention; half-split pairs rotated on a head's first elements; keys seen within
  chunks of positions only; a learned sink a head in the softmax's denominator; a sigmoid gate for every element of the result.
* ``parallel``: softmax attention and a gated delta rule side by side, summed with a weight each.  The attention sees every
  earlier key; its q, k and v pass short convolutions ahead of the rotation; a sink, one sigmoid gate a head.  The delta rule
  has one decay a head.
* ``lightning``: linear attention with a fixed decay a head; silu on q, k and v; the heads normed together, a sigmoid gate.

The feed-forward is gated, gate and up held to a limit.  The stream starts as the token's vector times a factor.  A run of
layers is passed through several times with the same weights, every pass with caches and state of its own; a pass starts from
W [x; x0] (x0 the embedding's output) plus a vector of the pass.  A final norm, an untied head.  Tensor names: ``embed``,
``head``, ``final.norm``, ``loop.in``, ``loop.step`` and per layer ``l<i>.norm1``, ``l<i>.mix.*``, ``l<i>.mlp.*``.
"""
from __future__ import annotations

from ..config.sonulorn import LightningConfig, SinkAttentionConfig, SonulornConfig
from ..parts.base import PartSpec
from ..parts.model import LayerRun, ModelSpec, StreamJoin
from .registry import register_architecture


def _norm(config: SonulornConfig, name: str) -> PartSpec:
    return PartSpec("rmsnorm", {"size": config.width, "eps": config.eps, "weight": name})


def _attention(config: SonulornConfig, m: SinkAttentionConfig, p: str, positions: dict, gate_each: bool) -> PartSpec:
    position = None
    if m.rot_dims is not None:
        position = f"rope_{m.rot_dims}_{m.rot_base!r}"
        positions.setdefault(position, PartSpec("rope_half_split", {"rotary_dim": m.rot_dims, "theta": m.rot_base}))
    params = {"hidden": config.width, "q_heads": m.heads, "kv_heads": m.kv_heads, "head_dim": m.dim, "value_dim": m.vdim,
              "qk_norm_eps": None, "window": None, "chunk": m.chunk, "scale": m.scale, "position": position, "float_output": True,
              "q": p + "q", "k": p + "k", "v": p + "v", "o": p + "o", "sink": p + "sink", "gate": p + "g", "gate_each": gate_each}
    if m.taps is not None:
        params["conv"] = {"taps": m.taps, "q": p + "q.conv", "k": p + "k.conv", "v": p + "v.conv"}
    return PartSpec("gqa_attention", params)


def _mixer(config: SonulornConfig, i: int, positions: dict) -> PartSpec:
    m, p = config.layers[i].mixer, f"l{i}.mix."
    if isinstance(m, SinkAttentionConfig):
        return _attention(config, m, p, positions, gate_each=True)
    if isinstance(m, LightningConfig):
        return PartSpec("retention", {"hidden": config.width, "heads": m.heads, "dim": m.dim, "vdim": m.vdim, "decay": list(m.decay),
                                      "eps": config.eps, "position": None, "activation": "silu", "k_scale": 1.0,
                                      "norm_span": "heads", "gate": "sigmoid", "q": p + "q", "k": p + "k", "v": p + "v",
                                      "g": p + "g", "o": p + "o", "norm": p + "norm"})
    r, y = m.right, p + "right."
    right = PartSpec("head_delta", {"hidden": config.width, "heads": r.heads, "kv_heads": r.kv_heads, "dim": r.dim, "vdim": r.vdim,
                                    "taps": r.taps, "eps": config.eps, "q": y + "q", "k": y + "k", "v": y + "v",
                                    "q_conv": y + "q.conv", "k_conv": y + "k.conv", "v_conv": y + "v.conv", "b": y + "b",
                                    "a": y + "a", "A_log": y + "A_log", "dt_bias": y + "dt_bias", "g": y + "g",
                                    "norm": y + "norm", "o": y + "o"})
    return PartSpec("parallel", {"hidden": config.width, "eps": config.eps,
                                 "branches": {"left": _attention(config, m.left, p + "left.", positions, gate_each=False),
                                              "right": right},
                                 "weights": {"left": m.left_scale, "right": m.right_scale}})


def layer_order(config: SonulornConfig) -> list:
    """(layer, the number of the pass that begins with it or None), one entry for every layer run."""
    n, loop = len(config.layers), config.loop
    if loop is None:
        return [(i, None) for i in range(n)]
    passes = [(i, t if i == loop.start else None) for t in range(loop.times) for i in range(loop.start, loop.stop)]
    return [(i, None) for i in range(loop.start)] + passes + [(i, None) for i in range(loop.stop, n)]


def sonulorn_model_spec(config: SonulornConfig) -> ModelSpec:
    positions: dict = {}
    layers = []
    for i, layer in enumerate(config.layers):
        p = f"l{i}."
        params = {"hidden": config.width, "norm1": _norm(config, p + "norm1"), "mixer": _mixer(config, i, positions)}
        if layer.mlp is not None:
            params["feed_forward"] = PartSpec("swiglu", {
                "hidden": config.width, "intermediate": layer.mlp.ff, "gate": p + "mlp.gate", "up": p + "mlp.up",
                "down": p + "mlp.down", "activation": "clamped_swish", "limit": layer.mlp.limit, "float_output": True})
        layers.append(PartSpec("parallel_prenorm", params))
    order = layer_order(config)
    join = None
    if config.loop is not None:
        join = StreamJoin(tuple(at for at, (_, begins) in enumerate(order) if begins is not None), "loop.in", "loop.step")
    return ModelSpec(hidden_size=config.width, vocab_size=config.vocab, max_positions=config.max_positions,
                     embedding="embed", layers=layers,
                     # every run, also of a layer that runs again, keeps a cache of its own
                     schedule=[LayerRun(layer, at) for at, (layer, _) in enumerate(order)],
                     final_norm=_norm(config, "final.norm"), head="head", positions=positions,
                     embedding_scale=config.embedding_scale, join=join)


register_architecture(SonulornConfig.ARCHITECTURE, SonulornConfig.from_dict, sonulorn_model_spec)
