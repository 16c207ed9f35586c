"""Reverax: how its configuration becomes parts.

A small decoder-only design whose config.json lists its layers one by one.  A layer's mixer and feed-forward read the same
stream through norms of their own and are added together (``parallel_prenorm`` block), each result times a learned vector:
x <- x + ls1 * mixer(norm1(x)) + ls2 * ff(norm2(x)).  The norms are RMS norms in equal groups of columns.  Two mixers:

* ``attention``: grouped-query softmax attention, projections with biases, neighbouring pairs rotated on a head's first
  elements, the heads' scaled scores mixed by a learned matrix before the softmax, every earlier key in sight.
* ``parallel``: softmax attention and a matrix memory (RWKV) side by side, summed with a weight each.  The attention has
  biases, q and k normed per head, half-split pairs rotated, values that turn with their own position and are turned back
  at the position that reads them, capped scores, a learned sink in the denominator and a window.  The memory reads the
  token before beside the token itself and makes its decays per key channel from it.

The feed-forward is gated with silu, or a mixture of ungated experts (squared relu) whose router takes the ``top`` largest
sigmoid scores and multiplies what an expert reads by its score.  The head is the token table, logits times
``logit_scale``.  A layer may take another layer's weights; it keeps a cache of its own.  Tensor names: ``embed``,
``final.norm`` and per layer ``l<i>.norm1``, ``l<i>.norm2``, ``l<i>.ls1``, ``l<i>.ls2``, ``l<i>.mix.*``, ``l<i>.mlp.*``.
"""
from __future__ import annotations

from ..config.reverax import DenseConfig, ReveraxConfig, TalkingAttentionConfig
from ..parts.base import PartSpec
from ..parts.model import LayerRun, ModelSpec
from .registry import register_architecture


def _norm(config: ReveraxConfig, name: str, factor: float = 1.0) -> PartSpec:
    params = {"size": config.width, "eps": config.eps, "weight": name, "groups": config.norm_groups}
    if factor != 1.0:
        params["gain_factor"] = factor
    return PartSpec("rmsnorm", params)


def _rope(kind: str, dims: int, base: float, positions: dict) -> str:
    name = f"{kind}_{dims}_{base!r}"
    positions.setdefault(name, PartSpec(kind, {"rotary_dim": dims, "theta": base}))
    return name


def _attention(config: ReveraxConfig, m, p: str) -> dict:
    return {"hidden": config.width, "q_heads": m.heads, "kv_heads": m.kv_heads, "head_dim": m.dim, "value_dim": m.vdim,
            "scale": m.scale, "float_output": True, "q": p + "q", "k": p + "k", "v": p + "v", "o": p + "o",
            "bias": {"q": p + "q.b", "k": p + "k.b", "v": p + "v.b"}}


def _mixer(config: ReveraxConfig, i: int, positions: dict) -> PartSpec:
    m, p = config.layers[i].mixer, f"l{i}.mix."
    if isinstance(m, TalkingAttentionConfig):
        return PartSpec("gqa_attention", {**_attention(config, m, p), "qk_norm_eps": None, "window": None, "talk": p + "talk",
                                          "position": _rope("rope_adjacent", m.rot_dims, m.rot_base, positions)})
    l, r = m.left, m.right
    x, y = p + "left.", p + "right."
    if r.decay_rank is None:
        raise ValueError(f"layer {i}: the decay's rank comes with the tensors (ReveraxConfig.with_shapes or with_ranks)")
    left = PartSpec("gqa_attention", {
        **_attention(config, l, x), "qk_norm_eps": config.eps, "q_norm": x + "q.norm", "k_norm": x + "k.norm",
        "window": l.window, "softcap": l.softcap, "sink": x + "sink",
        "position": _rope("rope_half_split", l.rot_dims, l.rot_base, positions),
        "value_position": _rope("rope_half_split", l.vdim, l.rot_base, positions)})
    names = {n: y + n for n in ("r", "k", "v", "g", "o", "norm", "u", "w0", "w1", "w2")}
    right = PartSpec("time_mix", {"hidden": config.width, "heads": r.heads, "dim": r.dim, "rank": r.decay_rank,
                                  "eps": config.eps, "mu": {n: y + "mu." + n for n in ("r", "k", "v", "g", "w")}, **names})
    return PartSpec("parallel", {"hidden": config.width, "eps": config.eps, "branches": {"left": left, "right": right},
                                 "weights": {"left": m.left_scale, "right": m.right_scale}})


def _feed_forward(config: ReveraxConfig, i: int):
    f, p = config.layers[i].mlp, f"l{i}.mlp."
    if f is None:
        return None
    if isinstance(f, DenseConfig):
        return PartSpec("swiglu", {"hidden": config.width, "intermediate": f.ff, "gate": p + "gate", "up": p + "up",
                                   "down": p + "down", "float_output": True})
    return PartSpec("routed_glu", {"hidden": config.width, "experts": f.experts, "identity": 0, "top": f.top,
                                   "group_count": 1, "group_keep": 1, "intermediate": f.expert_ff, "activation": "relu2",
                                   "gated": False, "score": "sigmoid", "renormalize": False, "weigh_input": True,
                                   "router": p + "router", "correction": None, "expert": p + "e{e}", "shared": None})


def reverax_model_spec(config: ReveraxConfig) -> ModelSpec:
    positions: dict = {}
    layers, unused, place = [], [], {}
    for i, layer in enumerate(config.layers):
        if layer.weights_of is not None:
            continue                            # runs another layer's parts
        p = f"l{i}."
        params = {"hidden": config.width, "norm1": _norm(config, p + "norm1"), "mixer": _mixer(config, i, positions),
                  "scale1": p + "ls1"}
        feed_forward = _feed_forward(config, i)
        if feed_forward is not None:
            params.update(norm2=_norm(config, p + "norm2"), feed_forward=feed_forward, scale2=p + "ls2")
        else:                                   # a file may hold what would belong to the sublayer that is not there
            unused += [p + "norm2", p + "ls2"]
        place[i] = len(layers)
        layers.append(PartSpec("parallel_prenorm", params))
    schedule = [LayerRun(place[i if layer.weights_of is None else layer.weights_of], i) for i, layer in enumerate(config.layers)]
    return ModelSpec(hidden_size=config.width, vocab_size=config.vocab, max_positions=config.max_positions,
                     embedding="embed", layers=layers, schedule=schedule,
                     # the logits' factor rides on the final norm's gain
                     final_norm=_norm(config, "final.norm", config.logit_scale), head=None, positions=positions,
                     ignore_tensors=tuple(unused))


register_architecture(ReveraxConfig.ARCHITECTURE, ReveraxConfig.from_dict, reverax_model_spec)
