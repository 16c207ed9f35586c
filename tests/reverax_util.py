"""Small Reverax configurations and weights for the tests, made here from the design's naming alone (the product's
list of tensors is checked against this, not used to make it)."""
from __future__ import annotations

import json
import math
import os
from typing import Dict

import numpy as np
import torch


def attention(heads, kv_heads, dim, vdim, dims, base=1000.0, scale=None):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                      "scale": scale if scale is not None else dim ** -0.5, "rot": {"dims": dims, "base": base}}}


def parallel(left, right, left_scale=0.5, right_scale=0.5, scale=None):
    """``left`` = (heads, kv_heads, dim, vdim, rotated elements, base, mask, cap), ``right`` = (heads, dim)."""
    heads, kv_heads, dim, vdim, dims, base, mask, cap = left
    l = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5,
         "rot": {"dims": dims, "base": base}}
    if cap is not None:
        l["softcap"] = cap
    if mask is not None:
        l["mask"] = {"size": mask}
    return {"type": "parallel", "mixer": {"left": l, "right": dict(zip(("heads", "dim"), right)), "left_scale": left_scale,
                                          "right_scale": right_scale}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def layer(mixer, mlp=None):
    return {**mixer, "mlp": mlp}


def config(width, vocab, layers, eps=1e-5, groups=1, logit_scale=1.0, max_positions=1024):
    return {"architecture": "Reverax", "vocab": vocab, "width": width, "norm": {"eps": eps, "groups": groups},
            "logit_scale": logit_scale, "max_positions": max_positions, "layers": layers}


def again(layers, *which):
    """The layers with copies behind them that take the weights of the layers named."""
    return layers + [{**layers[j], "weights_of": j} for j in which]


# Sizes unlike one another: one key/value head, several, and as many as query heads; keys and values of different sizes;
# rotated parts that are a piece of a head and the whole; windows below, at and above a page of 16, of one key, and none;
# capped scores and not; memories of one head and several, of sizes that fill no lane evenly; norms in one group and
# several, of sizes that are no multiples of 4; every mixer first, last and between; layers without feed-forward; routers
# that take one expert, several and all; layers that take another's weights, twice over, ahead of and behind it.
SMALL = {
    "A": config(64, 211, again([
        layer(parallel((4, 2, 16, 24, 8, 100.0, 20, 5.0), (3, 8), 0.8, -0.6), moe(6, 2, 24)),
        layer(attention(4, 2, 16, 24, 8, 500.0), dense(40)),
        layer(parallel((2, 1, 24, 8, 24, 10000.0, None, None), (1, 40), 1.3, 0.4), None),
        layer(attention(3, 3, 8, 8, 8), moe(4, 1, 16)),
    ], 0, 1), groups=4, logit_scale=1.7),
    "B": config(90, 130, again([
        layer(attention(6, 1, 16, 32, 4, 77.0), moe(5, 5, 8)),
        layer(parallel((6, 3, 16, 16, 16, 77.0, 16, 30.0), (2, 24), 0.7, 1.25), dense(24)),
        layer(attention(1, 1, 40, 16, 16, 30000.0), None),
        layer(parallel((5, 5, 8, 16, 2, 20.0, 1, 2.0), (4, 12), -0.5, 0.9), moe(7, 3, 16)),
    ], 1, 3, 1), eps=1e-6, groups=9, logit_scale=0.6),
    "C": config(128, 257, [
        layer(attention(8, 2, 32, 32, 16), moe(16, 4, 32)),
        layer(parallel((8, 1, 32, 32, 16, 1000.0, 24, 20.0), (4, 32), 1.0, 1.0), moe(8, 2, 64)),
        {**layer(parallel((4, 4, 64, 64, 32, 1000.0, 50, 8.0), (2, 64), 0.5, 1.1), dense(96)), "weights_of": 3},
        layer(parallel((4, 4, 64, 64, 32, 1000.0, 50, 8.0), (2, 64), 0.5, 1.1), dense(96)),
        layer(attention(16, 4, 32, 32, 32), dense(96)),
    ], groups=2, logit_scale=2.5),
}


def rank_of(i):
    """The rank of layer i's low-rank decay: another one for every layer."""
    return (8, 5, 16, 12, 3)[i % 5]


def tensor_shapes(raw: dict) -> Dict[str, tuple]:
    w, shapes = raw["width"], {}
    shapes["embed"] = (raw["vocab"], w)
    for i, entry in enumerate(raw["layers"]):
        if entry.get("weights_of") is not None:
            continue
        p, m, f = f"l{i}.", entry["mixer"], entry["mlp"]
        shapes.update({p + "norm1": (w,), p + "ls1": (w,)})

        def heads(x, a):
            qw, kw, vw = a["heads"] * a["dim"], a["kv_heads"] * a["dim"], a["kv_heads"] * a["vdim"]
            shapes.update({x + "q": (qw, w), x + "q.b": (qw,), x + "k": (kw, w), x + "k.b": (kw,), x + "v": (vw, w),
                           x + "v.b": (vw,), x + "o": (w, a["heads"] * a["vdim"])})
        x = p + "mix."
        if entry["type"] == "attention":
            heads(x, m)
            shapes[x + "talk"] = (m["heads"], m["heads"])
        else:
            l, r = m["left"], m["right"]
            heads(x + "left.", l)
            shapes.update({x + "left.q.norm": (l["dim"],), x + "left.k.norm": (l["dim"],), x + "left.sink": (l["heads"],)})
            y, inner, rank = x + "right.", r["heads"] * r["dim"], r.get("decay_rank", rank_of(i))
            shapes.update({y + "mu." + n: (w,) for n in ("r", "k", "v", "g", "w")})
            shapes.update({y + n: (inner, w) for n in ("r", "k", "v", "g")})
            shapes.update({y + "w1": (rank, w), y + "w2": (inner, rank), y + "w0": (inner,), y + "u": (r["heads"], r["dim"]),
                           y + "norm": (inner,), y + "o": (w, inner)})
        if f is None:
            continue
        shapes.update({p + "norm2": (w,), p + "ls2": (w,)})
        y = p + "mlp."
        if f["kind"] == "dense":
            shapes.update({y + "gate": (f["ff"], w), y + "up": (f["ff"], w), y + "down": (w, f["ff"])})
        else:
            shapes[y + "router"] = (f["router"]["experts"], w)
            for e in range(f["router"]["experts"]):
                shapes.update({f"{y}e{e}.up": (f["expert"]["ff"], w), f"{y}e{e}.down": (w, f["expert"]["ff"])})
    shapes["final.norm"] = (w,)
    return shapes


def one_tensor(name: str, shape: tuple, gen, sharpen: float = 1.0) -> torch.Tensor:
    """Values at which the mechanism a tensor belongs to matters: projections that keep activations of order 1, biases of
    order 1/2, sinks on both sides of the scores, a score mix with large entries off its diagonal, token mixes between
    either token, decays that reach from a few tokens to hundreds back, a router whose outputs spread.  ``sharpen``
    scales the query projections, so that scores spread and a misplaced key moves the result."""
    parts = name.split(".")
    last = parts[-1]
    if last in ("norm1", "norm2", "norm"):
        return 1.0 + 0.2 * torch.randn(shape, generator=gen)
    if last in ("ls1", "ls2"):
        return 0.5 + 0.3 * torch.randn(shape, generator=gen)
    if last == "b":
        return 0.5 * torch.randn(shape, generator=gen)
    if last == "sink":
        return 1.0 + torch.randn(shape, generator=gen)
    if last == "talk":
        return 0.6 * torch.eye(shape[0]) + 0.5 * torch.randn(shape, generator=gen)
    if len(parts) > 1 and parts[-2] == "mu":
        return torch.rand(shape, generator=gen) * 1.4 - 0.2
    if last == "w0":
        return torch.rand(shape, generator=gen) * 7.0 - 6.0
    if last == "u":
        return torch.randn(shape, generator=gen)
    if last == "router":
        return torch.randn(shape, generator=gen) * (3.0 / math.sqrt(shape[-1]))
    if last == "q":
        return torch.randn(shape, generator=gen) * (1.5 * sharpen / math.sqrt(shape[-1]))
    if last in ("gate", "up"):
        return torch.randn(shape, generator=gen) * (2.5 / math.sqrt(shape[-1]))
    return torch.randn(shape, generator=gen) * (1.5 / math.sqrt(shape[-1]))


def make_weights(raw: dict, seed: int, dtype=torch.bfloat16, sharpen: float = 1.0) -> Dict[str, torch.Tensor]:
    gen = torch.Generator().manual_seed(seed)
    return {name: one_tensor(name, shape, gen, sharpen).to(dtype) for name, shape in tensor_shapes(raw).items()}


def write_dir(path: str, raw: dict, weights: Dict[str, torch.Tensor]) -> str:
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as handle:
        json.dump(raw, handle)
    save_file({k: v.contiguous() for k, v in weights.items()}, os.path.join(path, "model.safetensors"))
    return path


def relative_error(have: np.ndarray, want: np.ndarray) -> np.ndarray:
    """Per row: root mean square of the difference (its mean taken off, as a logit's shift means nothing) over
    the root mean square of the expected logits."""
    d = have.astype(np.float64) - want.astype(np.float64)
    d = d - d.mean(axis=-1, keepdims=True)
    scale = np.sqrt((want.astype(np.float64) ** 2).mean()) + 1e-30
    return np.sqrt((d * d).mean(axis=-1)) / scale
