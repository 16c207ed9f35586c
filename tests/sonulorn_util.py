"""Small Sonulorn configurations and weights for the tests, made here from the design's naming alone (the product's
list of tensors is checked against this, not used to make it)."""
from __future__ import annotations

import math
from typing import Dict

import torch

from tests.reverax_util import relative_error, write_dir  # noqa: F401  (the tests' own helpers)


def heads_config(heads, kv_heads, dim, vdim, dims, base=1000.0, scale=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5,
            "rot": {"dims": dims, "base": base}}


def attention(heads, kv_heads, dim, vdim, dims, chunk, base=1000.0, scale=None):
    return {"type": "attention", "mixer": {**heads_config(heads, kv_heads, dim, vdim, dims, base, scale), "mask": {"size": chunk}}}


def parallel(left, right, left_scale=0.5, right_scale=0.5, base=1000.0, scale=None):
    """``left`` = (heads, kv_heads, dim, vdim, rotated elements, taps), ``right`` = (heads, kv_heads, dim, vdim, taps)."""
    return {"type": "parallel",
            "mixer": {"left": {**heads_config(*left[:5], base, scale), "conv": left[5]},
                      "right": dict(zip(("heads", "kv_heads", "dim", "vdim", "conv"), right)),
                      "left_scale": left_scale, "right_scale": right_scale}}


def lightning(heads, dim, vdim, decay=None):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim,
                                           "decay": list(decay) if decay else [1.0 - 0.6 ** (h + 1) for h in range(heads)]}}


def dense(ff, limit=2.0):
    return {"kind": "dense", "ff": ff, "limit": limit}


def layer(mixer, mlp=None):
    return {**mixer, "mlp": mlp}


def config(width, vocab, layers, loop=None, eps=1e-5, embed_scale=1.0, max_positions=1024):
    out = {"architecture": "Sonulorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embed_scale},
           "max_positions": max_positions, "layers": layers}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


# Sizes unlike one another: one key/value head, several, and as many as query heads; keys and values of different sizes;
# rotated parts that are a piece of a head and the whole; chunks below, at and above a page of 16, of one position, and none
# that is reached; convolutions of 1 to 5 taps, other ones beside each other; memories of one head and several, of sizes that
# fill no lane evenly; decays of 0 and 1; every mixer first, last, inside and outside the loop; loops at the start, at the
# end, over one layer, run once and several times; layers without feed-forward.
SMALL = {
    "A": config(64, 211, [
        layer(attention(4, 2, 16, 24, 8, 20, 100.0), dense(40, 1.2)),
        layer(parallel((4, 1, 16, 24, 8, 4), (3, 3, 8, 12, 2), 0.8, -0.6, 500.0), dense(24, 0.7)),
        layer(lightning(3, 8, 20, (0.0, 0.95, 1.0)), None),
        layer(attention(2, 2, 24, 8, 24, 16), dense(56, 5.0)),
    ], (0, 3, 2), embed_scale=3.0),
    "B": config(90, 130, [
        layer(lightning(5, 24, 6), dense(30)),
        layer(lightning(1, 40, 16, (0.9,)), dense(17, 1.0)),
        layer(parallel((6, 3, 16, 16, 4, 1), (4, 2, 24, 10, 5), 1.3, 0.4, 77.0), None),
        layer(attention(6, 1, 16, 32, 2, 33, 30000.0), dense(44, 3.0)),
        layer(attention(1, 1, 40, 16, 16, 1), dense(20)),
        layer(parallel((5, 5, 8, 14, 8, 2), (2, 1, 12, 30, 1), -0.5, 0.9), dense(52, 0.4)),
    ], (2, 5, 3), eps=1e-6, embed_scale=0.5),
    "C": config(128, 257, [
        layer(parallel((8, 2, 32, 32, 16, 3), (4, 1, 32, 32, 3), 0.7, 1.2), dense(96, 1.5)),
        layer(lightning(4, 32, 64), dense(96)),
        layer(attention(8, 2, 64, 64, 32, 50), dense(128, 7.0)),
        layer(attention(16, 4, 32, 32, 32, 24), None),
    ], (3, 4, 4), embed_scale=8.0),
}


def tensor_shapes(raw: dict) -> Dict[str, tuple]:
    w, shapes = raw["width"], {}
    shapes["embed"] = (raw["vocab"], w)
    if raw.get("loop"):
        shapes.update({"loop.in": (w, 2 * w), "loop.step": (raw["loop"]["times"], w)})
    for i, entry in enumerate(raw["layers"]):
        p, m, f = f"l{i}.", entry["mixer"], entry["mlp"]
        shapes[p + "norm1"] = (w,)

        def qkv(x, a, q_heads, k_heads, v_heads, conv=None):
            sizes = {"q": q_heads * a["dim"], "k": k_heads * a["dim"], "v": v_heads * a["vdim"]}
            shapes.update({x + n: (size, w) for n, size in sizes.items()})
            if conv is not None:
                shapes.update({x + n + ".conv": (size, conv) for n, size in sizes.items()})
        x = p + "mix."
        if entry["type"] == "lightning":
            h, inner = m["heads"], m["heads"] * m["vdim"]
            qkv(x, m, h, h, h)
            shapes.update({x + "g": (inner, w), x + "o": (w, inner), x + "norm": (inner,)})
        elif entry["type"] == "attention":
            qkv(x, m, m["heads"], m["kv_heads"], m["kv_heads"])
            shapes.update({x + "sink": (m["heads"],), x + "g": (m["heads"] * m["vdim"], w), x + "o": (w, m["heads"] * m["vdim"])})
        else:
            l, r, y, z = m["left"], m["right"], x + "left.", x + "right."
            qkv(y, l, l["heads"], l["kv_heads"], l["kv_heads"], l["conv"])
            shapes.update({y + "sink": (l["heads"],), y + "g": (l["heads"], w), y + "o": (w, l["heads"] * l["vdim"])})
            qkv(z, r, r["kv_heads"], r["kv_heads"], r["heads"], r["conv"])
            inner = r["heads"] * r["vdim"]
            shapes.update({z + "b": (r["heads"], w), z + "a": (r["heads"], w), z + "A_log": (r["heads"],), z + "dt_bias": (r["heads"],),
                           z + "norm": (r["vdim"],), z + "g": (inner, w), z + "o": (w, inner)})
        if f is not None:
            y = p + "mlp."
            shapes.update({y + "gate": (f["ff"], w), y + "up": (f["ff"], w), y + "down": (w, f["ff"])})
    shapes.update({"final.norm": (w,), "head": (raw["vocab"], w)})
    return shapes


def one_tensor(name: str, shape: tuple, gen, sharpen: float = 1.0) -> torch.Tensor:
    """Values at which the mechanism a tensor belongs to matters: projections that keep activations of order 1, filters whose
    every tap counts, sinks on both sides of the scores, decays from a few tokens to hundreds, gates and ups beyond their limit,
    pass vectors of order 1/2.  ``sharpen`` scales the attention's query projections, so that scores spread and a misplaced key
    moves the result."""
    parts = name.split(".")
    last = parts[-1]
    if last in ("norm1", "norm"):
        return 1.0 + 0.2 * torch.randn(shape, generator=gen)
    if last == "conv":
        return torch.randn(shape, generator=gen) / math.sqrt(shape[-1]) + 0.3
    if last == "sink":
        return 1.0 + torch.randn(shape, generator=gen)
    if last == "A_log":
        return torch.rand(shape, generator=gen) * 2.0 - 1.0
    if last == "dt_bias":
        return torch.rand(shape, generator=gen) * 5.0 - 6.0
    if name == "loop.step":
        return 0.5 * torch.randn(shape, generator=gen)
    if last == "q":
        return torch.randn(shape, generator=gen) * (1.5 * sharpen / math.sqrt(shape[-1]))
    if last in ("gate", "up"):
        return torch.randn(shape, generator=gen) * (2.5 / math.sqrt(shape[-1]))
    return torch.randn(shape, generator=gen) * (1.5 / math.sqrt(shape[-1]))


def make_weights(raw: dict, seed: int, dtype=torch.bfloat16, sharpen: float = 1.0) -> Dict[str, torch.Tensor]:
    gen = torch.Generator().manual_seed(seed)
    return {name: one_tensor(name, shape, gen, sharpen).to(dtype) for name, shape in tensor_shapes(raw).items()}
