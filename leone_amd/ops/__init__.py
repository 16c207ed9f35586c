"""Tensor-level wrappers over the HIP entry points.

Each wrapper checks device, type, shape and contiguity on the host before the
launch, because a kernel that reads outside its operands can take the whole
GPU down.  Tensors must live on the GPU: there is no CPU path.
"""
from __future__ import annotations

from typing import Optional

import ctypes
import functools
import math
import threading
import weakref

import numpy as np
import torch

from . import profile
from .library import KernelError, call, library

F32, BF16 = 0, 1
_CODES = {torch.float32: F32, torch.bfloat16: BF16}


def _code(t: torch.Tensor, what: str) -> int:
    try:
        return _CODES[t.dtype]
    except KeyError:
        raise KernelError(f"{what}: element type {t.dtype} is not float32 or bfloat16") from None


def _dev(t: Optional[torch.Tensor], what: str, dtype=None, shape=None) -> int:
    """Checks one operand and returns its device address (0 for None)."""
    if t is None:
        return 0
    if not t.is_cuda:
        raise KernelError(f"{what}: tensor is on {t.device}; the kernels run on the GPU only")
    if not t.is_contiguous():
        raise KernelError(f"{what}: tensor must be contiguous")
    if dtype is not None and t.dtype != dtype:
        raise KernelError(f"{what}: expected {dtype}, found {t.dtype}")
    if shape is not None and tuple(t.shape) != tuple(shape):
        raise KernelError(f"{what}: expected shape {tuple(shape)}, found {tuple(t.shape)}")
    return t.data_ptr()


_raw_stream = getattr(torch._C, "_cuda_getCurrentRawStream", None)


_held = threading.local()                # .stream inside ``one_stream``: the handle that was current when it began


def _stream() -> int:
    """The current stream's handle.  Asked for before every launch, so the short way is taken where this
    torch has it (a tenth of the time of building a Stream object); within ``one_stream`` it was asked for once."""
    held = getattr(_held, "stream", None)
    if held is not None:
        return held
    if _raw_stream is not None:
        return _raw_stream(torch.cuda.current_device())
    return torch.cuda.current_stream().cuda_stream


class one_stream:
    """Within this context every launch of this thread goes to the stream that is current at its beginning: the
    few hundred launches of a step need not ask for it one by one (0.4 ms of the 4 ms the host takes to issue a
    step of the 8B shape).  Whoever changes the current stream inside (a graph capture does) opens a context of
    its own.  The handle is kept per thread, as torch keeps the current stream: engines that step side by side
    in threads of their own, each on its stream, do not see each other's."""

    def __enter__(self):
        self._before = getattr(_held, "stream", None)
        _held.stream = None
        _held.stream = _stream()
        return self

    def __exit__(self, *exc):
        _held.stream = self._before
        return False


def cache_dims_kv(k_pool: torch.Tensor, v_pool: torch.Tensor):
    """(pages, kv_heads, page_tokens, head_dim, value_dim) of a key/value pool pair in the packed cache layout:
    keys ``[pages, kv_heads, head_dim/8, page_tokens, 8]``, values ``[pages, kv_heads, page_tokens/8, value_dim, 8]``."""
    if k_pool.dim() != 5 or k_pool.shape[4] != 8:
        raise KernelError(f"key pool must be [pages, kv_heads, head_dim/8, page_tokens, 8], found {tuple(k_pool.shape)}")
    pages, kv_heads, d8, page_tokens, _ = k_pool.shape
    if page_tokens % 8 or v_pool.dim() != 5 or (tuple(v_pool.shape[:3]) + (v_pool.shape[4],)) != (pages, kv_heads, page_tokens // 8, 8):
        raise KernelError(f"value pool must be [pages, kv_heads, page_tokens/8, value_dim, 8] matching the key pool "
                          f"{tuple(k_pool.shape)}, found {tuple(v_pool.shape)}")
    return pages, kv_heads, page_tokens, d8 * 8, v_pool.shape[3]


def cache_dims(k_pool: torch.Tensor, v_pool: torch.Tensor):
    """(pages, kv_heads, page_tokens, head_dim) of a pool pair whose values have the keys' size."""
    pages, kv_heads, page_tokens, head_dim, value_dim = cache_dims_kv(k_pool, v_pool)
    if value_dim != head_dim:
        raise KernelError(f"values of {value_dim} elements beside keys of {head_dim}: this kernel takes one size for both")
    return pages, kv_heads, page_tokens, head_dim


def pack_keys(k: torch.Tensor) -> torch.Tensor:
    """[..., tokens, head_dim] -> the packed page layout [..., head_dim/8, tokens, 8]."""
    *lead, tokens, dim = k.shape
    return k.reshape(*lead, tokens, dim // 8, 8).transpose(-3, -2).contiguous()


def pack_values(v: torch.Tensor) -> torch.Tensor:
    """[..., tokens, head_dim] -> the packed page layout [..., tokens/8, head_dim, 8]."""
    *lead, tokens, dim = v.shape
    return v.reshape(*lead, tokens // 8, 8, dim).transpose(-2, -1).contiguous()


def embed(table: torch.Tensor, tokens: torch.Tensor, out: Optional[torch.Tensor] = None,
          scale: float = 1.0, position_table: Optional[torch.Tensor] = None,
          positions: Optional[torch.Tensor] = None, copy: Optional[torch.Tensor] = None) -> torch.Tensor:
    """out[r] = table[tokens[r]] * scale as float32.  Token ids must have been checked against the table.  ``copy`` (float32
    ``[rows, hidden]``) receives the same rows once more.
    With ``position_table`` ``[places, hidden]`` (a learned vector for every position, of the table's type)
    row r also gets position_table[positions[r]], unscaled; the caller checks positions against ``places``."""
    vocab, hidden = table.shape
    rows = tokens.numel()
    if out is None:
        out = torch.empty((rows, hidden), dtype=torch.float32, device=table.device)
    if position_table is not None:
        if positions is None or position_table.dtype != table.dtype or position_table.dim() != 2 or position_table.shape[1] != hidden:
            raise KernelError(f"embed: a position table {tuple(position_table.shape)} {position_table.dtype} beside a token "
                              f"table {tuple(table.shape)} {table.dtype} needs the rows' positions and the same type and width")
        call("leone_embed_placed", _dev(table, "embed table"), _code(table, "embed table"),
             _dev(tokens, "embed tokens", torch.int32, (rows,)), _dev(out, "embed out", torch.float32, (rows, hidden)),
             rows, hidden, vocab, float(scale), _dev(position_table, "position table"),
             _dev(positions, "positions", torch.int32, (rows,)), position_table.shape[0],
             _dev(copy, "embed copy", torch.float32, (rows, hidden)), _stream())
        return out
    call("leone_embed_placed", _dev(table, "embed table"), _code(table, "embed table"),
         _dev(tokens, "embed tokens", torch.int32, (rows,)), _dev(out, "embed out", torch.float32, (rows, hidden)),
         rows, hidden, vocab, float(scale), 0, 0, 0, _dev(copy, "embed copy", torch.float32, (rows, hidden)), _stream())
    return out


def soft_cap(x: torch.Tensor, cap: float) -> torch.Tensor:
    """x = cap * tanh(x / cap), in place (float32)."""
    call("leone_soft_cap", _dev(x, "soft_cap values", torch.float32), x.numel(), float(cap), _stream())
    return x


def add_rmsnorm(x: torch.Tensor, delta: Optional[torch.Tensor], gain: torch.Tensor, eps: float,
                out_dtype: torch.dtype, rows: Optional[torch.Tensor] = None,
                out: Optional[torch.Tensor] = None, prepare: bool = False):
    """x += delta, then y = rmsnorm(x) * gain; with ``rows``, y[i] comes from row rows[i] and x is not written.
    ``delta`` is [n, hidden] or a stack of planes [p, n, hidden] whose sum, taken in order, is meant (the
    parts of a product whose inner dimension was cut, see ``linear``).  With ``prepare`` the norm is left for
    the product that consumes it to finish: ``PreparedRows`` comes back (the operand x * gain, and the rows'
    sums of squares), which rounds where the product with the norm folded in rounds."""
    n, hidden = x.shape
    n_out = n if rows is None else rows.numel()
    if out is None:
        out = torch.empty((n_out, hidden), dtype=out_dtype, device=x.device)
    squares = torch.empty((n_out, -(-hidden // 16)), dtype=torch.float32, device=x.device) if prepare else None
    delta_code = _code(delta, "add_rmsnorm delta") if delta is not None else _CODES[out_dtype]
    stacked = delta is not None and delta.dim() == 3
    planes = delta.shape[0] if stacked else 1
    if not 1 <= planes <= 16:
        raise KernelError(f"add_rmsnorm: {planes} planes of what is to be added")
    call("leone_add_rmsnorm", _dev(x, "add_rmsnorm x", torch.float32),
         _dev(delta, "add_rmsnorm delta", None, (planes, n, hidden) if stacked else (n, hidden)), delta_code, planes,
         n * hidden,
         _dev(gain, "add_rmsnorm gain", None, (hidden,)), _code(gain, "add_rmsnorm gain"), float(eps),
         _dev(out, "add_rmsnorm out", out_dtype, (n_out, hidden)), _CODES[out_dtype],
         _dev(rows, "add_rmsnorm rows", torch.int32), n_out, hidden, _dev(squares, "add_rmsnorm sums"), _stream())
    return PreparedRows(x, gain, eps, out_dtype, out, squares, rows) if prepare else out


GATE_ACTIVATIONS = {"silu": 0, "gelu_tanh": 1}     # what a gated feed-forward puts on its gate
# ... and what stands on gate and up together: "clamped_swish" holds both to a limit (see ``glu_value``)
GLU_ACTIVATIONS = {**GATE_ACTIVATIONS, "clamped_swish": 2}


def _gate_code(activation: str) -> int:
    try:
        return GATE_ACTIVATIONS[activation]
    except KeyError:
        raise KernelError(f"unknown gate activation {activation!r}; known: {', '.join(GATE_ACTIVATIONS)}") from None


def _glu_code(activation: str, limit: Optional[float]) -> int:
    code = GLU_ACTIVATIONS.get(activation)
    if code is None:
        raise KernelError(f"unknown gate activation {activation!r}; known: {', '.join(GLU_ACTIVATIONS)}")
    if code == 2 and not (limit is not None and limit > 0.0):
        raise KernelError(f"the clamped activation needs a positive limit, found {limit!r}")
    return code


def swiglu(gate_up: torch.Tensor, out: Optional[torch.Tensor] = None, activation: str = "silu",
           limit: Optional[float] = None) -> torch.Tensor:
    """act(gate) * up of rows that hold 8 gates, their 8 ups, and so on; ``activation`` names act (``GLU_ACTIVATIONS``), ``limit``
    belongs to "clamped_swish" alone."""
    rows, twice = gate_up.shape
    if twice % 2:
        raise KernelError("swiglu: input width must be even (gate columns, then up columns)")
    ffn = twice // 2
    if out is None:
        out = torch.empty((rows, ffn), dtype=gate_up.dtype, device=gate_up.device)
    call("leone_glu", _dev(gate_up, "swiglu in"), _dev(out, "swiglu out", gate_up.dtype, (rows, ffn)),
         _code(gate_up, "swiglu in"), rows, ffn, _glu_code(activation, limit), float(limit or 0.0), _stream())
    return out


def rope_table(theta: float, rotary_dim: int, positions: int, device) -> tuple[torch.Tensor, torch.Tensor]:
    cos = torch.empty((positions, rotary_dim // 2), dtype=torch.float32, device=device)
    sin = torch.empty_like(cos)
    call("leone_rope_table", _dev(cos, "rope cos"), _dev(sin, "rope sin"), float(theta), rotary_dim, positions,
         _stream())
    return cos, sin


PAIRINGS = {"half_split": 0, "adjacent": 1}   # which two elements of a head a rotation turns together


def _rotation_shape(what: str, head_dim: int, cos, sin, pairing: str):
    """(table positions, rotary_dim, pairing code) of a rotation given as cos/sin tables ``[positions,
    rotary_dim / 2]``: the head's first ``rotary_dim`` elements are rotated, in pairs (i, i + rotary_dim / 2)
    ("half_split") or (2 i, 2 i + 1) ("adjacent") (crates/leone/src/cpu.rs:1765-1774); the rest is left as it is."""
    if pairing not in PAIRINGS:
        raise KernelError(f"{what}: unknown pairing {pairing!r}; known: {', '.join(PAIRINGS)}")
    if cos is None:
        return 0, 0, PAIRINGS[pairing]
    if sin is None or sin.shape != cos.shape or cos.dim() != 2:
        raise KernelError(f"{what}: cos and sin tables must both be [positions, rotary_dim / 2]")
    rotary_dim = 2 * cos.shape[1]
    if not 0 < rotary_dim <= head_dim:
        raise KernelError(f"{what}: the rotary tables cover {rotary_dim} elements, a head has {head_dim}")
    return cos.shape[0], rotary_dim, PAIRINGS[pairing]


def decode_projected_supported(head_dim: int, rotary_dim: int = 0, pairing: str = "half_split") -> bool:
    """Whether ``attention_decode_projected`` takes this head and rotation: head sizes that are multiples of
    64, no rotation (``rotary_dim`` 0) or the half-split one over the whole head."""
    return head_dim % 64 == 0 and (rotary_dim == 0 or (rotary_dim == head_dim and pairing == "half_split"))


def qk_norm_rope_write(qkv: torch.Tensor, q_heads: int, kv_heads: int, head_dim: int,
                       q_gain: Optional[torch.Tensor], k_gain: Optional[torch.Tensor], eps: float,
                       cos: Optional[torch.Tensor], sin: Optional[torch.Tensor], positions: torch.Tensor,
                       row_entry: Optional[torch.Tensor], block_table: Optional[torch.Tensor],
                       k_pool: Optional[torch.Tensor], v_pool: Optional[torch.Tensor], write_cache: bool = True,
                       out: Optional[torch.Tensor] = None, out_dtype: Optional[torch.dtype] = None,
                       pairing: str = "half_split", value_dim: Optional[int] = None,
                       queries_only: bool = False, bias: Optional[torch.Tensor] = None,
                       value_rotation: Optional[tuple] = None, norm_count: int = 0) -> torch.Tensor:
    """Splits the fused projection, normalises and rotates q and k heads, writes k and v into the cache.
    ``qkv`` is ``[rows, width]`` of the cache's type, or float32 (also as planes ``[p, rows, width]`` whose
    sum, in order, is meant: a product cut along K) with ``out_dtype`` naming the type of q and the cache.
    The rotation's shape comes with its tables (``_rotation_shape``): their width says how much of a head is
    rotated, ``pairing`` which elements go together.  ``value_dim``: the value heads' own size (then a row may
    also hold further columns behind the heads, which are left alone).  ``queries_only``: the rows hold the query
    heads (and perhaps further columns) but no key and value heads: a layer that reads another layer's cache.
    ``bias`` (a vector over all heads' columns) is added first.  ``value_rotation`` = (cos, sin, pairing): value heads
    are turned by their own position over their whole size before they are cached.  ``norm_count``: only so many
    elements of a head exist (the rest are zeros that do not count in the heads' norms; 0: all)."""
    planes = qkv.shape[0] if qkv.dim() == 3 else 1
    rows, width = qkv.shape[-2:]
    kind = out_dtype or qkv.dtype
    if qkv.dtype != kind and qkv.dtype != torch.float32:
        raise KernelError(f"qk_norm_rope_write: input {qkv.dtype} for outputs of {kind}")
    general = value_dim is not None
    value_dim = head_dim if value_dim is None else int(value_dim)
    heads_width = (q_heads + kv_heads) * head_dim + kv_heads * value_dim
    if queries_only:
        if write_cache or planes != 1 or width < q_heads * head_dim:
            raise KernelError(f"qk_norm_rope_write: rows of {width} with query heads only ({q_heads}*{head_dim}) write no cache")
    elif width != heads_width and not (general and width > heads_width and planes == 1):
        raise KernelError(f"qk_norm_rope_write: width {width} is not ({q_heads}+{kv_heads})*{head_dim}+{kv_heads}*{value_dim}")
    if out is None:
        out = torch.empty((rows, q_heads * head_dim), dtype=kind, device=qkv.device)
    max_blocks = page_tokens = 0
    if write_cache:
        if k_pool is None or v_pool is None or block_table is None or row_entry is None:
            raise KernelError("qk_norm_rope_write: a cache write needs pools, a block table and a row map")
        pages, pool_heads, page_tokens, pool_dim, pool_vdim = cache_dims_kv(k_pool, v_pool)
        if (pool_heads, pool_dim, pool_vdim) != (kv_heads, head_dim, value_dim):
            raise KernelError(f"qk_norm_rope_write: pool shapes {tuple(k_pool.shape)}, {tuple(v_pool.shape)} do not fit "
                              f"{kv_heads} heads of {head_dim} and {value_dim}")
        max_blocks = block_table.shape[1]
    table_positions, rotary_dim, pairing_code = _rotation_shape("qk_norm_rope_write", head_dim, cos, sin, pairing)
    gain_code = _code(q_gain, "q gain") if q_gain is not None else F32
    if q_gain is not None and (k_gain is None or k_gain.dtype != q_gain.dtype):
        raise KernelError("qk_norm_rope_write: q and k gains must come together in one type")
    v_cos = v_sin = None
    v_positions = v_pairing = 0
    if value_rotation is not None:
        v_cos, v_sin = value_rotation[:2]
        v_positions, v_dims, v_pairing = _rotation_shape("qk_norm_rope_write values", value_dim, v_cos, v_sin, value_rotation[2])
        if v_dims != value_dim:
            raise KernelError(f"qk_norm_rope_write: values of {value_dim} elements are turned whole, the tables cover {v_dims}")
    if not 0 <= norm_count <= head_dim:
        raise KernelError(f"qk_norm_rope_write: {norm_count} of {head_dim} elements in a head's norm")
    if bias is not None and bias.numel() != (q_heads * head_dim if queries_only else heads_width):
        raise KernelError(f"qk_norm_rope_write: a bias of {bias.numel()} for heads of {heads_width} columns")
    call("leone_qk_norm_rope_write_turned", _dev(qkv, "qkv"), _code(qkv, "qkv"), planes, rows * width,
         _dev(out, "q out", kind),
         _dev(k_pool if write_cache else None, "k pool", kind),
         _dev(v_pool if write_cache else None, "v pool", kind), _CODES[kind],
         _dev(q_gain, "q gain", None, (head_dim,)), _dev(k_gain, "k gain", None, (head_dim,)), gain_code,
         float(eps), _dev(cos, "rope cos", torch.float32), _dev(sin, "rope sin", torch.float32), table_positions,
         rotary_dim, pairing_code, _dev(positions, "positions", torch.int32, (rows,)),
         _dev(row_entry if write_cache else None, "row map", torch.int32, (rows,)),
         _dev(block_table if write_cache else None, "block table", torch.int32), max_blocks, rows, q_heads,
         kv_heads, head_dim, page_tokens, 1 if write_cache else 0, value_dim, width, _dev(bias, "bias"),
         _code(bias, "bias") if bias is not None else F32, _dev(v_cos, "value cos", torch.float32),
         _dev(v_sin, "value sin", torch.float32), v_positions, v_pairing, int(norm_count), _stream())
    return out


class ScoreShape:
    """What an attention does to its scores and results beside the mask: ``cap`` (scaled scores become cap * tanh(score /
    cap)), ``sinks`` (float32 ``[q_heads]``: exp(sinks[h]) stands in the denominator and weighs no value) and ``turn`` =
    (cos, sin, pairing): the cached values were turned by their positions, a row's results are turned back by its own
    (tables float32 ``[positions, value size / 2]``)."""

    def __init__(self, cap: Optional[float] = None, sinks: Optional[torch.Tensor] = None, turn: Optional[tuple] = None):
        self.cap, self.sinks, self.turn = float(cap or 0.0), sinks, turn

    def args(self, q_heads: int, value_dim: int) -> tuple:
        cos, sin, pairing = self.turn if self.turn is not None else (None, None, "half_split")
        positions, dims, code = _rotation_shape("attention results", value_dim, cos, sin, pairing)
        if cos is not None and dims != value_dim:
            raise KernelError(f"attention: results of {value_dim} elements are turned back whole, the tables cover {dims}")
        return (self.cap, _dev(self.sinks, "sinks", torch.float32, (q_heads,)), _dev(cos, "turn cos", torch.float32),
                _dev(sin, "turn sin", torch.float32), positions, code)


_PLAIN_SCORES = ScoreShape()


def _strided_rows(t: Optional[torch.Tensor], what: str, rows: int, columns: int, dtype=torch.float32):
    """(address, elements from row to row) of a 2-D float view whose rows may be slices of wider rows."""
    if t is None:
        return 0, 0
    if not t.is_cuda or t.dtype != dtype or t.dim() != 2 or t.shape[0] != rows or t.shape[1] < columns \
            or (t.shape[1] > 1 and t.stride(1) != 1) or t.stride(0) < t.shape[1]:
        raise KernelError(f"{what}: expected {dtype} [{rows}, >= {columns}] with unit stride along a row, found "
                          f"{t.dtype} {tuple(t.shape)} strides {t.stride()} on {t.device}")
    return t.data_ptr(), t.stride(0)


def attention_rows(q: torch.Tensor, k_pool: torch.Tensor, v_pool: torch.Tensor, positions: torch.Tensor,
                   row_entry: torch.Tensor, block_table: torch.Tensor, q_heads: int, scale: float,
                   window: int = 0, out: Optional[torch.Tensor] = None, gate: Optional[torch.Tensor] = None,
                   keep_first: int = 0, gate_each: bool = False, slopes: Optional[torch.Tensor] = None,
                   query_factor: Optional[tuple] = None, shape: Optional[ScoreShape] = None, chunk: int = 0) -> torch.Tensor:
    """Each query row attends its request's cached keys up to its own position (the last ``window`` of them,
    and, whatever the window, those at positions below ``keep_first``).  The result has the values'
    size a head.  ``slopes`` float32 ``[q_heads]``: head h's score for the key at distance d is lowered by
    slopes[h] * d.  ``query_factor`` = (coef, every): the queries of a row at position p count times
    1 + coef * ln(floor((p + 1) / every) + 1).  ``gate``: float32 ``[rows, >= q_heads]`` (a view into a wider row is fine, unit stride along the
    heads): head h of row r is multiplied by sigmoid(gate[r, h]); with ``gate_each`` the gate holds a value for
    every element of the result, ``[rows, >= q_heads * value_dim]``.  ``shape``: capped scores, sinks, results turned
    back (``ScoreShape``; results are turned back before the gate).  ``chunk`` (without a window): a row sees the keys of its
    own chunk of so many positions, counted from 0, only."""
    rows = q.shape[0]
    pages, kv_heads, page_tokens, head_dim, value_dim = cache_dims_kv(k_pool, v_pool)
    if q.shape[1] != q_heads * head_dim:
        raise KernelError(f"attention: query width {q.shape[1]} is not {q_heads}*{head_dim}")
    if out is None:
        out = torch.empty((rows, q_heads * value_dim), dtype=q.dtype, device=q.device)
    gate_at, gate_stride = _strided_rows(gate, "attention gate", rows, q_heads * value_dim if gate_each else q_heads)
    coef, every = query_factor if query_factor is not None else (0.0, 0)
    call("leone_attention_rows_shaped", _dev(q, "attention q"), _dev(out, "attention out", q.dtype, (rows, q_heads * value_dim)),
         _dev(k_pool, "k pool", q.dtype), _dev(v_pool, "v pool", q.dtype), _code(q, "attention q"),
         _dev(positions, "positions", torch.int32, (rows,)), _dev(row_entry, "row map", torch.int32, (rows,)),
         _dev(block_table, "block table", torch.int32), block_table.shape[1], rows, q_heads, kv_heads, head_dim,
         value_dim, page_tokens, float(scale), int(window), gate_at, gate_stride, int(keep_first),
         1 if (gate_each and gate is not None) else 0, _dev(slopes, "slopes", torch.float32, (q_heads,)), float(coef),
         int(every), *(shape or _PLAIN_SCORES).args(q_heads, value_dim), int(chunk), _stream())
    return out


def attention_rows_talk(q: torch.Tensor, k_pool: torch.Tensor, v_pool: torch.Tensor, talk: torch.Tensor, positions: torch.Tensor,
                        row_entry: torch.Tensor, block_table: torch.Tensor, q_heads: int, scale: float, window: int = 0,
                        out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``attention_rows`` whose heads' scaled scores are mixed before the softmax: score_h <- sum_g talk[h, g] score_g over
    all query heads g (``talk`` ``[q_heads, q_heads]``).  Any type and size."""
    rows = q.shape[0]
    pages, kv_heads, page_tokens, head_dim, value_dim = cache_dims_kv(k_pool, v_pool)
    if q.shape[1] != q_heads * head_dim:
        raise KernelError(f"attention: query width {q.shape[1]} is not {q_heads}*{head_dim}")
    if out is None:
        out = torch.empty((rows, q_heads * value_dim), dtype=q.dtype, device=q.device)
    call("leone_attention_rows_talk", _dev(q, "attention q"), _dev(out, "attention out", q.dtype, (rows, q_heads * value_dim)),
         _dev(k_pool, "k pool", q.dtype), _dev(v_pool, "v pool", q.dtype), _code(q, "attention q"),
         _dev(talk, "talk", None, (q_heads, q_heads)), _code(talk, "talk"), _dev(positions, "positions", torch.int32, (rows,)),
         _dev(row_entry, "row map", torch.int32, (rows,)), _dev(block_table, "block table", torch.int32), block_table.shape[1],
         rows, q_heads, kv_heads, head_dim, value_dim, page_tokens, float(scale), int(window), _stream())
    return out


TALK_TILE_ROWS = 16            # rows of a tile of ``attention_talk_prefill`` (checked against the library)
TALK_MIN_ROWS = 16             # portions from so many rows on go there


def talk_attention_supported(dtype: torch.dtype, q_heads: int, head_dim: int, value_dim: int, page_tokens: int, max_blocks: int = 0) -> dict:
    """Which matrix-core kernels for mixed scores take this shape: {"decode": ..., "prompt": ...}; the others go to
    ``attention_rows_talk``.  The prompt kernel's workgroup holds 16 rows' queries of every head in shared memory, which
    leaves room for the numbers of 2,560 pages."""
    fits = (dtype == torch.bfloat16 and head_dim % 8 == 0 and value_dim % 4 == 0 and max(head_dim, value_dim) <= 128
            and page_tokens >= 16 and page_tokens & (page_tokens - 1) == 0 and 4 * max_blocks <= 32 * 1024)
    return {"decode": fits and q_heads <= 32, "prompt": fits and q_heads <= 32 and max_blocks <= 2560}


def _talk_operands(q, k_pool, v_pool, talk, q_heads: int):
    rows = q.shape[0]
    pages, kv_heads, page_tokens, head_dim, value_dim = cache_dims_kv(k_pool, v_pool)
    if q.shape[1] != q_heads * head_dim:
        raise KernelError(f"attention: query width {q.shape[1]} is not {q_heads}*{head_dim}")
    _dev(talk, "talk", None, (q_heads, q_heads))
    return rows, kv_heads, page_tokens, head_dim, value_dim


def attention_talk_decode(q: torch.Tensor, k_pool: torch.Tensor, v_pool: torch.Tensor, talk: torch.Tensor, positions: torch.Tensor,
                          row_entry: torch.Tensor, block_table: torch.Tensor, q_heads: int, scale: float, window: int = 0,
                          max_context: int = 1, splits: Optional[int] = None, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``attention_rows_talk`` on the matrix cores (bfloat16; ``talk_attention_supported``), a row's keys cut into
    ``splits`` parts.  ``max_context`` only steers their number."""
    rows, kv_heads, page_tokens, head_dim, value_dim = _talk_operands(q, k_pool, v_pool, talk, q_heads)
    if splits is None:
        reach = min(max_context, window + 32) if window else max_context
        splits = choose_splits(rows, 1, 1, reach, compute_units(q.device))     # one workgroup takes all heads of a row
    if out is None:
        out = torch.empty((rows, q_heads * value_dim), dtype=torch.bfloat16, device=q.device)
    part_acc = part_ml = None
    if splits > 1:
        part_acc = torch.empty((rows * q_heads * splits * value_dim,), dtype=torch.float32, device=q.device)
        part_ml = torch.empty((rows * q_heads * splits * 2,), dtype=torch.float32, device=q.device)
    call("leone_attention_talk_decode", _dev(q, "attention q", torch.bfloat16),
         _dev(out, "attention out", torch.bfloat16, (rows, q_heads * value_dim)), _dev(k_pool, "k pool", torch.bfloat16),
         _dev(v_pool, "v pool", torch.bfloat16), _dev(talk, "talk"), _code(talk, "talk"),
         _dev(positions, "positions", torch.int32, (rows,)), _dev(row_entry, "row map", torch.int32, (rows,)),
         _dev(block_table, "block table", torch.int32), block_table.shape[1], _dev(part_acc, "partials"), _dev(part_ml, "partial sums"),
         rows, q_heads, kv_heads, head_dim, value_dim, page_tokens, float(scale), int(window), int(splits), _stream())
    return out


def choose_talk_splits(tiles: int, mean_keys: int, units: int = 256) -> int:
    """Into how many parts the keys of a tile of rows are cut (a tile of more than 16 heads counts twice): the number for
    which rounds of workgroups (one a compute unit) x (stages of 64 keys a part + a start worth 3 + a merge worth 2) come
    out least."""
    stages = max(1, -(-mean_keys // 64))
    best = None
    for splits in range(1, min(16, stages) + 1):
        cost = (-(-tiles * splits // units) * (-(-stages // splits) + 3 + (2 if splits > 1 else 0)), splits)
        if best is None or cost < best:
            best = cost
    return best[1]


def attention_talk_prefill(q: torch.Tensor, out: torch.Tensor, k_pool: torch.Tensor, v_pool: torch.Tensor, talk: torch.Tensor,
                           positions: torch.Tensor, tiles: torch.Tensor, block_table: torch.Tensor, q_heads: int, scale: float,
                           mean_keys: int = 1, splits: Optional[int] = None, covered_rows: Optional[int] = None) -> torch.Tensor:
    """``attention_rows_talk`` without a window for the rows that ``tiles`` (int32 [n, 3]: entry, first row, up to
    TALK_TILE_ROWS consecutive rows of one request) covers; writes into ``out``."""
    if library().leone_attention_talk_tile_rows() != TALK_TILE_ROWS:
        raise KernelError("the kernel library was built for another tile size of mixed-score attention")
    rows, kv_heads, page_tokens, head_dim, value_dim = _talk_operands(q, k_pool, v_pool, talk, q_heads)
    if tiles.dim() != 2 or tiles.shape[1] != 3:
        raise KernelError(f"attention_talk_prefill: tiles must be int32 [n, 3], found {tuple(tiles.shape)}")
    if splits is None:
        splits = choose_talk_splits(tiles.shape[0] * (1 if q_heads <= 16 else 2), mean_keys, compute_units(q.device))
    part_acc = part_ml = None
    if splits > 1:
        covered = rows if covered_rows is None else covered_rows
        if not 0 < covered <= rows:
            raise KernelError(f"attention_talk_prefill: {covered} covered rows of {rows}")
        part_acc = torch.empty((covered * q_heads * splits * value_dim,), dtype=torch.float32, device=q.device)
        part_ml = torch.empty((covered * q_heads * splits * 2,), dtype=torch.float32, device=q.device)
    call("leone_attention_talk_prefill", _dev(q, "attention q", torch.bfloat16),
         _dev(out, "attention out", torch.bfloat16, (rows, q_heads * value_dim)), _dev(k_pool, "k pool", torch.bfloat16),
         _dev(v_pool, "v pool", torch.bfloat16), _dev(talk, "talk"), _code(talk, "talk"),
         _dev(positions, "positions", torch.int32, (rows,)), _dev(tiles, "tiles", torch.int32), tiles.shape[0],
         _dev(block_table, "block table", torch.int32), block_table.shape[1], _dev(part_acc, "partials"), _dev(part_ml, "partial sums"),
         q_heads, kv_heads, head_dim, value_dim, page_tokens, float(scale), int(splits), _stream())
    return out


def decode_attention_supported(dtype: torch.dtype, head_dim: int, page_tokens: int, group: int = 1,
                               max_blocks: int = 0) -> bool:
    """Whether the matrix-core kernel takes this case; otherwise ``attention_rows`` does."""
    cols = min(group, 16)
    shared = (4 * cols * head_dim + 8 * cols) * 4 + 4 * max_blocks   # the four waves' partial results, page ids
    return (dtype == torch.bfloat16 and head_dim % 16 == 0 and 16 <= head_dim <= 256 and shared <= 64 * 1024
            and page_tokens >= 16 and page_tokens & (page_tokens - 1) == 0)


DECODE_SPLIT_START_TILES = 8   # what starting a workgroup of the split-KV kernel costs, in 32-key tiles


def choose_splits(rows: int, kv_heads: int, group: int, max_context: int, units: int = 256) -> int:
    """Into how many parts the keys of a row are cut: the number (up to 32, at least four 32-key tiles a part,
    one for each of a workgroup's waves) for which the compute unit with the most workgroups has the least to
    do: ceil(workgroups / units) x (tiles a part + a start worth 8 tiles).  Measured in whole decode steps at
    8,192 keys, 1 to 48 rows, against a fixed aim of one or two workgroups a unit: level where those do well
    (1, 8, 12, 17 rows) and up to 15 % of a step better where their workgroup counts leave units idle or a few
    with one workgroup more than the rest (24 rows: 8.67 ms against 9.18, 40 rows: 11.8 against 13.9)."""
    blocks = rows * kv_heads * ((group + 15) // 16)
    tiles = (max_context + 31) // 32
    best = None
    for splits in range(1, min(32, max(1, tiles // 4)) + 1):
        cost = (-(-blocks * splits // units) * (-(-tiles // splits) + DECODE_SPLIT_START_TILES), splits)
        if best is None or cost < best:
            best = cost
    return best[1]


def attention_decode(q: torch.Tensor, k_pool: torch.Tensor, v_pool: torch.Tensor, positions: torch.Tensor,
                     row_entry: torch.Tensor, block_table: torch.Tensor, q_heads: int, scale: float,
                     window: int = 0, max_context: int = 1, splits: Optional[int] = None,
                     out: Optional[torch.Tensor] = None, keep_first: int = 0, slopes: Optional[torch.Tensor] = None,
                     query_factor: Optional[tuple] = None, shape: Optional[ScoreShape] = None, chunk: int = 0,
                     gate: Optional[torch.Tensor] = None, gate_each: bool = False) -> torch.Tensor:
    """Split-KV attention on the matrix cores (bfloat16).  ``max_context`` only steers the number of splits.
    ``keep_first``: keys at positions below it stay in sight of a windowed layer.  ``slopes`` and ``query_factor``
    as for ``attention_rows``: scores that fall with the distance, queries that count more the further on they stand.
    ``shape``: capped scores, sinks, results turned back.  ``chunk``, ``gate`` and ``gate_each`` as for ``attention_rows``."""
    rows = q.shape[0]
    pages, kv_heads, page_tokens, head_dim = cache_dims(k_pool, v_pool)
    if q.shape[1] != q_heads * head_dim:
        raise KernelError(f"attention: query width {q.shape[1]} is not {q_heads}*{head_dim}")
    gate_at, gate_stride = _strided_rows(gate, "attention gate", rows, q_heads * head_dim if gate_each else q_heads)
    if splits is None:
        reach = min(max_context, window + keep_first + 32) if window else max_context     # keys a row can see at most
        reach = min(reach, chunk) if chunk else reach
        splits = choose_splits(rows, kv_heads, q_heads // kv_heads, reach, compute_units(q.device))
    if out is None:
        out = torch.empty_like(q)
    part_acc = part_ml = None
    if splits > 1:
        part_acc = torch.empty((rows * q_heads * splits * head_dim,), dtype=torch.float32, device=q.device)
        part_ml = torch.empty((rows * q_heads * splits * 2,), dtype=torch.float32, device=q.device)
    coef, every = query_factor if query_factor is not None else (0.0, 0)
    call("leone_attention_decode_shaped", _dev(q, "attention q", torch.bfloat16),
         _dev(out, "attention out", torch.bfloat16, q.shape), _dev(k_pool, "k pool", torch.bfloat16),
         _dev(v_pool, "v pool", torch.bfloat16), _dev(positions, "positions", torch.int32, (rows,)),
         _dev(row_entry, "row map", torch.int32, (rows,)), _dev(block_table, "block table", torch.int32),
         block_table.shape[1], _dev(part_acc, "partials"), _dev(part_ml, "partial sums"), rows, q_heads, kv_heads,
         head_dim, page_tokens, float(scale), int(window), int(splits), int(keep_first) if window else 0,
         _dev(slopes, "slopes", torch.float32, (q_heads,)), float(coef), int(every),
         *(shape or _PLAIN_SCORES).args(q_heads, head_dim), int(chunk), gate_at, gate_stride, 1 if gate_each else 0, _stream())
    return out


def attention_decode_projected(qkv: torch.Tensor, q_heads: int, kv_heads: int, head_dim: int,
                               q_gain: Optional[torch.Tensor], k_gain: Optional[torch.Tensor], eps: float,
                               cos: Optional[torch.Tensor], sin: Optional[torch.Tensor], k_pool: torch.Tensor,
                               v_pool: torch.Tensor, positions: torch.Tensor, row_entry: torch.Tensor,
                               block_table: torch.Tensor, scale: float, window: int = 0, max_context: int = 1,
                               splits: Optional[int] = None, write_cache: bool = True,
                               pairing: str = "half_split") -> torch.Tensor:
    """``qk_norm_rope_write`` and ``attention_decode`` in one launch, for a step in which every row is another
    request (single decoded tokens): the kernel takes the fused q/k/v projection (bfloat16 ``[rows, width]``, or
    float32 planes ``[p, rows, width]``), makes queries and the new key itself and writes key and value into
    the cache before it reads the keys.  Head sizes that are multiples of 64."""
    planes = qkv.shape[0] if qkv.dim() == 3 else 1
    rows, width = qkv.shape[-2:]
    pages, pool_heads, page_tokens, pool_dim = cache_dims(k_pool, v_pool)
    if (pool_heads, pool_dim) != (kv_heads, head_dim) or width != (q_heads + 2 * kv_heads) * head_dim:
        raise KernelError(f"attention_decode_projected: width {width} and pool {tuple(k_pool.shape)} do not fit "
                          f"{q_heads}+2*{kv_heads} heads of {head_dim}")
    if head_dim % 64:
        raise KernelError(f"attention_decode_projected: head size {head_dim} is no multiple of 64")
    table_positions, rotary_dim, pairing_code = _rotation_shape("attention_decode_projected", head_dim, cos, sin, pairing)
    if not decode_projected_supported(head_dim, rotary_dim, pairing):
        raise KernelError(f"attention_decode_projected: the kernel rotates whole heads in half-split pairs, not "
                          f"{rotary_dim} of {head_dim} elements in {pairing} pairs (qk_norm_rope_write and "
                          f"attention_decode take those)")
    if q_gain is not None and (k_gain is None or k_gain.dtype != q_gain.dtype):
        raise KernelError("attention_decode_projected: q and k gains must come together in one type")
    if splits is None:
        splits = choose_splits(rows, kv_heads, q_heads // kv_heads, max_context, compute_units(qkv.device))
    out = torch.empty((rows, q_heads * head_dim), dtype=torch.bfloat16, device=qkv.device)
    part_acc = part_ml = None
    if splits > 1:
        part_acc = torch.empty((rows * q_heads * splits * head_dim,), dtype=torch.float32, device=qkv.device)
        part_ml = torch.empty((rows * q_heads * splits * 2,), dtype=torch.float32, device=qkv.device)
    call("leone_attention_decode_projected", _dev(qkv, "qkv"), _code(qkv, "qkv"), planes, rows * width,
         _dev(q_gain, "q gain", None, (head_dim,)), _dev(k_gain, "k gain", None, (head_dim,)),
         _code(q_gain, "q gain") if q_gain is not None else F32, float(eps),
         _dev(cos, "rope cos", torch.float32), _dev(sin, "rope sin", torch.float32), table_positions, rotary_dim,
         pairing_code, _dev(out, "attention out"), _dev(k_pool, "k pool", torch.bfloat16), _dev(v_pool, "v pool", torch.bfloat16),
         1 if write_cache else 0, _dev(positions, "positions", torch.int32, (rows,)),
         _dev(row_entry, "row map", torch.int32, (rows,)), _dev(block_table, "block table", torch.int32),
         block_table.shape[1], _dev(part_acc, "partials"), _dev(part_ml, "partial sums"), rows, q_heads, kv_heads,
         head_dim, page_tokens, float(scale), int(window), int(splits), _stream())
    return out


PREFILL_TILE_ROWS = 32       # rows of one request a wave of the prompt kernel takes (checked against the library)
PREFILL_GROUP_TILES = 4      # tiles of one request a workgroup of the prompt kernel takes (likewise)
PREFILL_MIN_ROWS = 16        # shorter portions go through the split-KV kernel row by row
PREFILL_MAX_SPLITS = 32      # most key ranges the prompt kernel takes (checked against the library)
PREFILL_SPLIT_MIN_STAGES = 4 # a key range of the prompt kernel keeps at least this many 64-key stages
PREFILL_SPLIT_START_STAGES = 8   # what a workgroup of the prompt kernel costs before its first stage, in stages
PREFILL_SPLIT_MERGE_STAGES = 6   # what writing and merging a range's partial results adds, in stages


def prefill_attention_supported(dtype: torch.dtype, head_dim: int, page_tokens: int, max_blocks: int = 0) -> bool:
    return (dtype == torch.bfloat16 and head_dim % 16 == 0 and 16 <= head_dim <= 128
            and 16 * max_blocks <= 64 * 1024                      # the page ids of four waves' keys
            and page_tokens >= 16 and page_tokens & (page_tokens - 1) == 0)


def choose_prefill_splits(groups: int, q_heads: int, mean_keys: int, window: int = 0, units: int = 256) -> int:
    """How many ranges the keys of a prompt workgroup are cut into, where a row sees ``mean_keys`` keys: the
    number (a range keeps at least PREFILL_SPLIT_MIN_STAGES stages of 64 keys) for which the rounds of
    workgroups over the chip (two fit a compute unit) x (stages a range + the start, + the merge where there
    is more than one range) come out least.  Measured in whole
    steps on portions of 128 to 1,536 rows after 30,720 positions against a fixed aim of two workgroups a unit:
    level for 256, 512 and 1,024 rows, 28.9 against 30.2 ms for 768 rows, 51.3 against 54.4 for 1,536.  (A
    prompt from position 0 gains nothing from ranges, its early rows see few keys: without the merge's term
    the rule took two ranges for 1,024 and 3,072 rows and lost 3 and 4 % of the step by it.)"""
    reach = PREFILL_GROUP_TILES * PREFILL_TILE_ROWS
    keys = min(mean_keys, window + reach) if window > 0 else mean_keys
    stages = -(-keys // 64)
    blocks = max(1, groups * q_heads)
    best = None
    for splits in range(1, min(PREFILL_MAX_SPLITS, max(1, stages // PREFILL_SPLIT_MIN_STAGES)) + 1):
        each = -(-stages // splits) + PREFILL_SPLIT_START_STAGES + (PREFILL_SPLIT_MERGE_STAGES if splits > 1 else 0)
        cost = (-(-blocks * splits // (2 * units)) * each, splits)
        if best is None or cost < best:
            best = cost
    return best[1]


def attention_prefill(q: torch.Tensor, out: torch.Tensor, k_pool: torch.Tensor, v_pool: torch.Tensor,
                      positions: torch.Tensor, tiles: torch.Tensor, block_table: torch.Tensor, q_heads: int,
                      scale: float, window: int = 0, mean_keys: int = 1, splits: Optional[int] = None,
                      covered_rows: Optional[int] = None, keep_first: int = 0, slopes: Optional[torch.Tensor] = None,
                      query_factor: Optional[tuple] = None, shape: Optional[ScoreShape] = None, chunk: int = 0) -> torch.Tensor:
    """Attention for the rows that ``tiles`` covers; writes into ``out``.  ``slopes``, ``query_factor``, ``shape`` and
    ``chunk`` as for ``attention_rows``.

    ``tiles`` is int32 [n, 3]: (entry, first row, rows) with at most PREFILL_TILE_ROWS consecutive rows of one
    request each, PREFILL_GROUP_TILES to a group, all tiles of a group of the same entry, unused places with
    0 rows (``prefill_tiles`` builds such a list).  ``mean_keys`` (keys a row sees on average) only steers
    the number of key ranges (``splits``); ``covered_rows``: one more than the last row a tile names, if the
    caller knows it.  ``keep_first``: keys at positions below it stay in sight of a windowed layer (the keys are
    then walked as one range)."""
    if (library().leone_attention_prefill_tile_rows() != PREFILL_TILE_ROWS
            or library().leone_attention_prefill_group_tiles() != PREFILL_GROUP_TILES
            or library().leone_attention_prefill_max_splits() != PREFILL_MAX_SPLITS):
        raise KernelError("the kernel library was built for another prompt tile size")
    rows = q.shape[0]
    pages, kv_heads, page_tokens, head_dim = cache_dims(k_pool, v_pool)
    if q.shape[1] != q_heads * head_dim:
        raise KernelError(f"attention: query width {q.shape[1]} is not {q_heads}*{head_dim}")
    if tiles.dim() != 2 or tiles.shape[1] != 3 or tiles.shape[0] % PREFILL_GROUP_TILES:
        raise KernelError(f"attention_prefill: tiles must be int32 [n, 3] with n a multiple of {PREFILL_GROUP_TILES}")
    groups = tiles.shape[0] // PREFILL_GROUP_TILES
    keep_first = int(keep_first) if window else 0
    if keep_first:
        splits = 1
    if splits is None:
        # a group's rows lie in one chunk or two
        splits = choose_prefill_splits(groups, q_heads, mean_keys, chunk or window, compute_units(q.device))
    part_acc = part_ml = None
    if splits > 1:
        covered = rows if covered_rows is None else covered_rows
        if not 0 < covered <= rows:
            raise KernelError(f"attention_prefill: {covered} covered rows of {rows}")
        part_acc = torch.empty((covered * q_heads * splits * head_dim,), dtype=torch.float32, device=q.device)
        part_ml = torch.empty((covered * q_heads * splits * 2,), dtype=torch.float32, device=q.device)
    coef, every = query_factor if query_factor is not None else (0.0, 0)
    call("leone_attention_prefill_shaped", _dev(q, "attention q", torch.bfloat16),
         _dev(out, "attention out", torch.bfloat16, q.shape), _dev(k_pool, "k pool", torch.bfloat16),
         _dev(v_pool, "v pool", torch.bfloat16), _dev(positions, "positions", torch.int32, (rows,)),
         _dev(tiles, "tiles", torch.int32), groups, _dev(block_table, "block table", torch.int32),
         block_table.shape[1], q_heads, kv_heads, head_dim, page_tokens, float(scale), int(window),
         _dev(part_acc, "partials"), _dev(part_ml, "partial sums"), int(splits), keep_first,
         _dev(slopes, "slopes", torch.float32, (q_heads,)), float(coef), int(every),
         *(shape or _PLAIN_SCORES).args(q_heads, head_dim), int(chunk), _stream())
    return out


def prefill_tiles(portions) -> torch.Tensor:
    """The tile list of ``attention_prefill`` for portions given as (entry, first row, rows): tiles in order,
    every portion's last group filled up with unused places (as the native step layout lists a step's own)."""
    tiles = []
    for entry, first_row, rows in portions:
        mine = [(entry, first_row + at, min(PREFILL_TILE_ROWS, rows - at)) for at in range(0, rows, PREFILL_TILE_ROWS)]
        mine += [(entry, first_row, 0)] * (-len(mine) % PREFILL_GROUP_TILES)
        tiles += mine
    return torch.tensor(tiles, dtype=torch.int32).view(-1, 3)


def gemm_f32(a: torch.Tensor, b: torch.Tensor, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """a[M,K] . b[N,K]^T in true single precision."""
    m, k = a.shape
    n, k2 = b.shape
    if k != k2:
        raise KernelError(f"gemm_f32: inner sizes {k} and {k2} differ")
    if out is None:
        out = torch.empty((m, n), dtype=torch.float32, device=a.device)
    with profile.span("gemm f32", b):
        call("leone_gemm_f32", _dev(a, "gemm a", torch.float32), _dev(b, "gemm b", torch.float32),
             _dev(out, "gemm out", torch.float32, (m, n)), m, n, k, _stream())
    return out


# Up to here norm, gate and residual are folded into the weight-streaming kernel for few rows; beyond, the
# multi-row kernel runs with the row-wise kernels between.  Measured in whole decode steps at the 8B layer sizes
# with the second copies of the weights (ms a step, folded : multi-row): 5.98 : 6.40 at 11 rows, 6.17 : 6.47 at
# 12, 6.51 : 6.66 at 14, level at 16, which is all the kernel takes.  (With row-major weights only, the folded
# kernel's reads of X weighed more and the two crossed between 10 and 11 rows.)
FUSED_ROWS = 16
FUSED_NORM_WEIGHT_ROWS = 1024   # a norm is folded into the product only for weights of at most this many rows


class NormedRows:
    """Rows of the float32 stream that are to be RMS-normalised: a norm not yet carried out, so that
    the product that consumes it can fold it in.  ``rows`` (int32 indices) picks rows of ``x``."""

    def __init__(self, x: torch.Tensor, gain: torch.Tensor, eps: float, dtype: torch.dtype,
                 rows: Optional[torch.Tensor] = None):
        self.x, self.gain, self.eps, self.dtype, self.rows = x, gain, float(eps), dtype, rows
        self.shape = (x.shape[0] if rows is None else rows.numel(), x.shape[1])

    def materialize(self) -> torch.Tensor:
        return add_rmsnorm(self.x, None, self.gain, self.eps, self.dtype, self.rows)

    def prepare(self) -> "PreparedRows":
        """The norm kernel runs, but leaves the scaling to the product (see ``add_rmsnorm``)."""
        return add_rmsnorm(self.x, None, self.gain, self.eps, self.dtype, self.rows, prepare=True)


class PreparedRows(NormedRows):
    """A norm of the stream ``x`` (of its rows ``rows``) whose operand lies ready: ``operand`` is
    bf16(x * gain), ``squares`` float32 ``[rows, ceil(hidden / 16)]`` partial sums of x^2.  The product before
    leaves them behind (``linear(..., next_norm=)``), so that the product that consumes them needs no norm
    kernel and no second read of the stream; or the norm kernel does (``add_rmsnorm(..., prepare=True)``).  The stream itself is
    up to date: any other consumer normalises it in the usual way (``materialize``)."""

    def __init__(self, x: torch.Tensor, gain: torch.Tensor, eps: float, dtype: torch.dtype,
                 operand: torch.Tensor, squares: torch.Tensor, rows: Optional[torch.Tensor] = None):
        super().__init__(x, gain, eps, dtype, rows)
        self.operand, self.squares = operand, squares


def prepared_fits(rows: int, hidden: int) -> bool:
    """Whether ``gemm_fused`` takes rows of this width as ``PreparedRows`` (its sums of squares travel in
    16-byte runs, at most 2,048 of them)."""
    return hidden % 64 == 0 and rows * (hidden // 64) <= 2048


def materialize(x) -> torch.Tensor:
    return x.materialize() if isinstance(x, NormedRows) else x


def interleave_gate_up(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
    """The fused gate/up weight: 8 gate rows, the 8 up rows that belong to them, and so on; the order in
    which ``swiglu`` and the gated product expect the columns of the product."""
    ffn, hidden = gate.shape
    if ffn % 8 or up.shape != gate.shape:
        raise KernelError(f"gate and up must both be [F, H] with F a multiple of 8, found {tuple(gate.shape)}")
    return torch.stack([gate.view(ffn // 8, 8, hidden), up.view(ffn // 8, 8, hidden)], dim=1).reshape(2 * ffn, hidden)


def tile_weight(weight: torch.Tensor) -> torch.Tensor:
    """The copy of ``weight[N, K]`` (bfloat16, K a multiple of 64) that the weight-streaming products read
    fastest: rows in tiles of 16 (the last filled up with zero rows), K in steps of 64, a step in two halves;
    element e of lane 16 g + c in half h of step s of tile t is ``weight[16 t + c][64 s + 16 g + 8 h + e]``, so
    ``[tiles, K / 64, 2, 4, 16, 8]``.  Each load of a wave is then 1 KB in one piece."""
    n, k = weight.shape
    if weight.dtype != torch.bfloat16 or k % 64:
        raise KernelError(f"tile_weight: a bfloat16 matrix with K a multiple of 64 is needed, not {weight.dtype} with K {k}")
    tiles = -(-n // 16)
    if tiles * 16 != n:
        weight = torch.cat([weight, weight.new_zeros((tiles * 16 - n, k))])
    return weight.view(tiles, 16, k // 64, 4, 2, 8).permute(0, 2, 4, 3, 1, 5).contiguous()


_streamed: dict = {}         # (address, shape) of a weight -> (weak reference to the weight, its tiled copy)


def keep_streamed_copy(weight: torch.Tensor) -> int:
    """Makes and keeps the tiled copy of a weight; the products take it from then on whenever they are given
    this weight, and it is dropped when the weight is.  Returns the copy's bytes (0 if the weight's shape or
    type has no tiled form)."""
    if weight.dtype != torch.bfloat16 or weight.dim() != 2 or weight.shape[1] % 64 or not weight.is_cuda:
        return 0
    key = (weight.data_ptr(), tuple(weight.shape))
    held = _streamed.get(key)
    if held is None or held[0]() is not weight:
        def forget(_, key=key):
            _streamed.pop(key, None)
        _streamed[key] = (weakref.ref(weight, forget), tile_weight(weight))
    return _streamed[key][1].numel() * 2


def streamed_copy(weight: torch.Tensor) -> Optional[torch.Tensor]:
    held = _streamed.get((weight.data_ptr(), tuple(weight.shape)))
    return None if held is None or held[0]() is not weight else held[1]


def drop_streamed_copies() -> None:
    _streamed.clear()


def gemm_fused(x, weight: torch.Tensor, out_dtype: torch.dtype = torch.bfloat16,
               residual: Optional[torch.Tensor] = None, gated: bool = False, next_norm=None, activation: str = "silu",
               limit: Optional[float] = None):
    """The product for at most 16 rows with its neighbours folded in: ``x`` may be ``NormedRows`` or
    ``PreparedRows``; with ``residual`` the product is added into that float32 tensor and None is returned;
    with ``gated`` the weight is an interleaved gate/up weight and silu(gate) * up comes out.  With
    ``residual`` and ``next_norm = (gain, eps, dtype)`` the kernel also leaves the operand of that norm
    behind and ``PreparedRows`` is returned (the residual has been added)."""
    m, k = x.shape
    n, k2 = weight.shape
    if k != k2:
        raise KernelError(f"gemm_fused: inner sizes {k} and {k2} differ")
    prepared = isinstance(x, PreparedRows)
    normed = isinstance(x, NormedRows) and not prepared
    if residual is not None and gated:
        raise KernelError("gemm_fused: a gated product cannot also be added into the stream")
    if next_norm is not None and residual is None:
        raise KernelError("gemm_fused: the next norm can only be prepared from the stream the product is added into")
    operand = squares = None
    if residual is not None:
        out, mode, out_dtype = residual, 1, torch.float32
        if next_norm is not None:
            mode = 3
            operand = torch.empty((m, n), dtype=torch.bfloat16, device=weight.device)
            squares = torch.empty((m, -(-n // 16)), dtype=torch.float32, device=weight.device)
    elif gated:
        # modes 4 and 5: the gated output with the tanh form of gelu on the gate, and with gate and up held to a limit
        out, mode, out_dtype = (torch.empty((m, n // 2), dtype=torch.bfloat16, device=weight.device),
                                (2, 4, 5)[_glu_code(activation, limit)], torch.bfloat16)
    else:
        out, mode = torch.empty((m, n), dtype=out_dtype, device=weight.device), 0
    if prepared:
        source, in_mode = _dev(x.operand, "prepared operand", torch.bfloat16, (m, k)), 2
        _dev(x.squares, "prepared sums", torch.float32, (m, -(-k // 16)))
    elif normed:
        source, in_mode = _dev(x.x, "stream", torch.float32), 1
    else:
        source, in_mode = _dev(x, "gemm x", torch.bfloat16, (m, k)), 0
    tiles = streamed_copy(weight) if _streamed else None
    with profile.span("gemv fused", weight):
        call("leone_gemm_fused_bf16", source, in_mode, _dev(x.rows, "rows", torch.int32) if normed else 0,
             _dev(x.gain, "gain", None, (k,)) if normed else 0, _code(x.gain, "gain") if normed else 0,
             x.eps if (normed or prepared) else 0.0,
             _dev(weight if tiles is None else tiles, "gemm weight", torch.bfloat16), 0 if tiles is None else 1,
             _dev(out, "gemm out", out_dtype, (m, n // 2 if gated else n)), mode, _CODES[out_dtype], m, n, k,
             x.squares.data_ptr() if prepared else 0, _dev(operand, "operand out"), _dev(squares, "sums out"),
             _dev(next_norm[0], "next gain", None, (n,)) if next_norm is not None else 0,
             _code(next_norm[0], "next gain") if next_norm is not None else 0, float(limit or 0.0), _stream())
    if next_norm is not None:
        return PreparedRows(residual, next_norm[0], next_norm[1], next_norm[2], operand, squares)
    return None if residual is not None else out


ROWS_MAX = 128               # most rows the multi-row weight-streaming product takes (checked against the library)
ROWS_WAVES = (4, 6, 8)       # workgroup sizes it is built for, in waves (16 weight rows each)
_UNITS = {}


def compute_units(device) -> int:
    index = torch.device(device).index or 0
    if index not in _UNITS:
        _UNITS[index] = torch.cuda.get_device_properties(index).multi_processor_count if torch.cuda.is_available() else 256
    return _UNITS[index]


def rows_plan(m: int, n: int, k: int, may_split: bool, units: int = 256) -> tuple[int, int]:
    """(waves, splits) for ``gemm_rows``: how many waves (tiles of 16 weight rows) a workgroup gets and into
    how many ranges K is cut.  The kernel is fastest with one workgroup on every compute unit and none
    waiting for a second round (6,144 x 4,096 at 64 rows: 18 us with 256 workgroups, 22 with 480, 24 with
    288), so the plan minimises rounds x the longest workgroup's traffic, where a chunk of K costs a
    workgroup its waves' weight tiles plus half of X's tiles (those come from the cache) and starting up
    costs as much as 3,072 elements of K; ties go to fewer ranges, then fewer waves.  The constants were set
    in whole decode steps of 17 to 128 rows at the layer sizes of the 8B, 14B and 32B models (a start of 768
    or 1,536 elements cuts long K's into too many ranges: 8B 8.05 : 7.91 ms a step at 64 rows; a fixed choice
    for matrices of many rows gave the 32B gate/up product 4 waves and four rounds where 8 waves need two:
    21.7 : 20.3 ms at 64 rows)."""
    return _rows_plan(m, n, k, bool(may_split), units, library().leone_gemm_rows_chunk(m), tuple(ROWS_WAVES))


@functools.lru_cache(maxsize=4096)
def _rows_plan(m: int, n: int, k: int, may_split: bool, units: int, chunk: int, waves_offered: tuple) -> tuple[int, int]:
    # the same few problems come back a few hundred times a step: 0.8 ms of a step's 4 on the host without this
    chunks = -(-k // chunk)
    tiles = -(-n // 16)
    x_tiles = -(-m // 16)
    best = None
    for waves in waves_offered:
        groups = -(-tiles // waves)
        for splits in range(1, (min(chunks, 16) if may_split else 1) + 1):
            per = -(-chunks // splits)
            if per * (splits - 1) >= chunks:            # a range would be empty
                continue
            rounds = -(-groups * splits // units)
            cost = (rounds * (per + 3072 // chunk) * (waves + 0.5 * x_tiles), splits, waves)
            if best is None or cost < best:
                best = cost
    return best[2], best[1]


ROWS_WAYS = 2                # most waves that share a tile of the weight in ``gemm_rows``


def rows_ways(m: int, waves: int) -> int:
    """How many waves share each tile of the weight in ``gemm_rows`` (each takes its share of a chunk's units of
    K; their sums are added up in a fixed order at the end): the most the kernel is built with for this many
    rows and tiles, up to ROWS_WAYS."""
    ways = ROWS_WAYS
    while ways > 1 and not library().leone_gemm_rows_shape_built(m, waves, ways):
        ways //= 2
    return ways


def gemm_rows(x: torch.Tensor, weight: torch.Tensor, out_dtype: torch.dtype = torch.bfloat16,
              residual: Optional[torch.Tensor] = None, gated: bool = False, splits: Optional[int] = None,
              waves: Optional[int] = None, may_split: bool = True, ways: Optional[int] = None,
              activation: str = "silu", tiles: Optional[torch.Tensor] = None,
              limit: Optional[float] = None) -> Optional[torch.Tensor]:
    """The weight-streaming product for up to ROWS_MAX rows of bfloat16 ``x``.  With ``residual`` and one
    range of K the product is added into that float32 tensor (None returned); with ``gated`` the weight is
    an interleaved gate/up weight and silu(gate) * up comes out.  With more than one range of K (``splits``;
    by default what ``rows_plan`` finds best, one if ``may_split`` is false or the product is gated) float32
    planes ``[splits, M, N]`` are returned whose sum, in order, is the product (with ``residual``: for the
    caller to add).  ``tiles``: the weight's second copy where it is not kept under the weight itself."""
    m, k = x.shape
    n, k2 = weight.shape
    if k != k2:
        raise KernelError(f"gemm_rows: inner sizes {k} and {k2} differ")
    if library().leone_gemm_rows_max_rows() != ROWS_MAX:
        raise KernelError("the kernel library was built for another number of rows")
    if not 1 <= m <= ROWS_MAX:
        raise KernelError(f"gemm_rows: {m} rows, the kernel takes 1..{ROWS_MAX}")
    if residual is not None and gated:
        raise KernelError("gemm_rows: a gated product cannot also be added into the stream")
    if splits is None or waves is None:
        plan = rows_plan(m, n, k, may_split and not gated, compute_units(weight.device))
        waves = plan[0] if waves is None else waves
        splits = plan[1] if splits is None else splits
    if ways is None:
        ways = rows_ways(m, int(waves))
    chunks = -(-k // library().leone_gemm_rows_chunk(m))
    splits = max(1, min(int(splits), chunks))
    splits = -(-chunks // -(-chunks // splits))        # no range of K may be empty
    if gated:
        splits = 1
    plane = 0
    if splits > 1:
        out, mode, kind = torch.empty((splits, m, n), dtype=torch.float32, device=weight.device), 3, torch.float32
        plane = m * n
    elif residual is not None:
        out, mode, kind = residual, 1, torch.float32
        _dev(out, "gemm_rows stream", torch.float32, (m, n))
    elif gated:
        out, mode, kind = (torch.empty((m, n // 2), dtype=torch.bfloat16, device=weight.device),
                           (2, 4, 5)[_glu_code(activation, limit)], torch.bfloat16)
    else:
        out, mode, kind = torch.empty((m, n), dtype=out_dtype, device=weight.device), 0, out_dtype
    if tiles is None and _streamed:
        tiles = streamed_copy(weight)
    with profile.span("gemm rows", weight):
        call("leone_gemm_rows_bf16", _dev(x, "gemm x", torch.bfloat16, (m, k)),
             _dev(weight if tiles is None else tiles, "gemm weight", torch.bfloat16), 0 if tiles is None else 1,
             _dev(out, "gemm out", kind), mode, _CODES[kind], m, n, k,
             splits, plane, int(waves), int(ways), float(limit or 0.0), _stream())
    return None if (residual is not None and splits == 1) else out


def inner_parts(rows: int, n: int, k: int) -> int:
    """Into how many parts the inner dimension of x[rows, k] . w[n, k]^T is cut when the result goes into the
    float32 stream.  The library's product does badly with a few hundred rows, few columns and a long inner
    dimension (the down projection of a prompt portion: 81 us whole against 64 in four parts for 512 x 4096 x
    12288, 171 against 97 for 512 x 5120 x 17408, 55 against 32 for 96 x 4096 x 12288); beyond 1,024 rows
    and up to 64 it is best left whole."""
    if not (64 < rows <= 1024 and k >= 8192 and k >= 2 * n):
        return 1
    for parts in ((4, 2) if rows <= 512 else (2,)):
        if k % (64 * parts) == 0:
            return parts
    return 1


# ---- the vendor library's product with a measured choice of its algorithm -------------------------------------
_tuned_products: set = set()     # (device index, m, n, k, output code, accumulate) of the problems tuned
_recorded_products = None        # while ``record_library_products`` runs: problem -> weights it was asked with


class record_library_products:
    """Within this context ``linear`` notes every product that it hands to the vendor library: the problem
    (rows, weight rows, inner size, output type, whether it adds into the stream) and the weights it came with.
    ``problems`` maps each problem to its weights afterwards."""

    def __enter__(self):
        global _recorded_products
        self.problems: dict = {}
        self._before = _recorded_products
        _recorded_products = self.problems
        return self

    def __exit__(self, *exc):
        global _recorded_products
        _recorded_products = self._before
        return False


def _library_problem(x: torch.Tensor, weight: torch.Tensor, out_dtype: torch.dtype, accumulate: bool):
    return (x.device.index or 0, x.shape[0], weight.shape[0], weight.shape[1], F32 if out_dtype == torch.float32 else BF16,
            1 if accumulate else 0)


def library_product_available() -> bool:
    return bool(library().leone_library_product_available())


def tune_library_product(rows: int, weights, out_dtype: torch.dtype, accumulate: bool, candidates: int = 256,
                         thorough: bool = False) -> dict:
    """Times the vendor library's algorithms for ``[rows, K] . W^T`` on ``weights`` (matrices of one shape, taken
    in turn as a model's layers are; ``candidates`` from the library's heuristic, with ``thorough`` every
    algorithm the library has) and keeps the fastest for ``linear`` to use on exactly this problem, after
    checking its result against a float32 product: it must be no further from it than twice what the library's
    ordinary call is.  Returns the problem, the microseconds of the library's own choice and of the winner, and
    how many algorithms were timed; ``kept`` is False if the winner failed the check and was dropped."""
    weights = list(weights)
    weight = weights[0]
    n, k = weight.shape
    if any(w.shape != weight.shape or w.dtype != torch.bfloat16 or not w.is_contiguous() for w in weights):
        raise KernelError("tune_library_product: the weights must be contiguous bfloat16 matrices of one shape")
    if accumulate and out_dtype != torch.float32:
        raise KernelError("tune_library_product: adding into the stream is a float32 product")
    generator = torch.Generator(device=weight.device).manual_seed(rows * 31 + n)
    x = torch.randn((rows, k), device=weight.device, generator=generator).to(torch.bfloat16)
    y = torch.zeros((rows, n), dtype=out_dtype, device=weight.device)
    import ctypes
    pointers = (ctypes.c_void_p * len(weights))(*[w.data_ptr() for w in weights])
    first, best, timed = ctypes.c_float(), ctypes.c_float(), ctypes.c_int()
    out_code = F32 if out_dtype == torch.float32 else BF16
    call("leone_library_product_tune", _dev(x, "x", torch.bfloat16), pointers, len(weights), _dev(y, "y"), rows, n, k,
         out_code, 1 if accumulate else 0, int(candidates), 1 if thorough else 0, ctypes.byref(first), ctypes.byref(best),
         ctypes.byref(timed), _stream())
    problem = _library_problem(x, weight, out_dtype, accumulate)
    # the check: the winner and the library's ordinary call against a float32 product, from a zero stream
    exact = torch.mm(x.float(), weight.float().t())
    y.zero_()
    call("leone_library_product", _dev(x, "x"), _dev(weight, "w"), _dev(y, "y"), rows, n, k, out_code,
         1 if accumulate else 0, _stream())
    usual = torch.mm(x, weight.t(), out_dtype=torch.float32) if out_dtype == torch.float32 else torch.nn.functional.linear(x, weight)
    off = (y.float() - exact).abs().max().item()
    usual_off = (usual.float() - exact).abs().max().item()
    kept = bool(off <= 2.0 * usual_off + 1e-6 * exact.abs().max().item())
    if kept:
        # An algorithm that reduces over K with atomics (split-K, stream-K) need not repeat bit for bit, and
        # then neither would the logits of a replayed trace: the winner runs again from the same zero stream,
        # and once more with the rows of x in reverse order (a row's bits must not depend on the other rows).
        again = torch.zeros_like(y)
        call("leone_library_product", _dev(x, "x"), _dev(weight, "w"), _dev(again, "y"), rows, n, k, out_code,
             1 if accumulate else 0, _stream())
        turned, x_turned = torch.zeros_like(y), x.flip(0).contiguous()
        call("leone_library_product", _dev(x_turned, "x"), _dev(weight, "w"), _dev(turned, "y"), rows, n, k, out_code,
             1 if accumulate else 0, _stream())
        kept = bool(torch.equal(again, y) and torch.equal(turned.flip(0), y))
    if kept:
        _tuned_products.add(problem)
    else:
        call("leone_library_product_forget", rows, n, k, out_code, 1 if accumulate else 0)
    return {"problem": problem, "rows": rows, "weight_rows": n, "inner": k, "float_out": out_dtype == torch.float32,
            "adds": bool(accumulate),
            "library_us": round(first.value, 1), "tuned_us": round(best.value, 1), "timed": timed.value, "kept": kept,
            "off": off, "library_off": usual_off}      # ``kept`` False: too far off, or not the same bits twice


def forget_tuned_products(problems=None) -> None:
    """Gives the named problems (all, if none are named) back to the library's heuristic."""
    for problem in list(_tuned_products if problems is None else problems):
        device, m, n, k, out_code, accumulate = problem
        with torch.cuda.device(device):
            call("leone_library_product_forget", m, n, k, out_code, accumulate)
        _tuned_products.discard(problem)


def _library_product(x: torch.Tensor, weight: torch.Tensor, out_dtype: torch.dtype,
                     residual: Optional[torch.Tensor]) -> Optional[torch.Tensor]:
    """The vendor library's product for many rows: bfloat16 or float32 out, or added into the float32 stream
    (then nothing comes back).  A problem that was tuned runs with the algorithm that won; any other goes
    through torch's call of the same library."""
    problem = _library_problem(x, weight, out_dtype, residual is not None)
    if _recorded_products is not None:
        known = _recorded_products.setdefault(problem[1:], [])
        if all(w is not weight for w in known):
            known.append(weight)
    if problem in _tuned_products and x.is_contiguous() and weight.is_contiguous():
        y = residual if residual is not None else torch.empty((x.shape[0], weight.shape[0]), dtype=out_dtype, device=x.device)
        call("leone_library_product", _dev(x, "x", torch.bfloat16), _dev(weight, "w", torch.bfloat16),
             _dev(y, "y", out_dtype, (x.shape[0], weight.shape[0])), x.shape[0], weight.shape[0], weight.shape[1],
             problem[4], problem[5], _stream())
        return None if residual is not None else y
    if residual is not None:
        # the library adds into the stream itself (float product plus float stream, the same bits as adding the
        # product afterwards), which saves the next norm's kernel the read of the product: 27.2 against 27.8 ms
        # for a prompt of 2,048 tokens
        torch.addmm(residual, x, weight.t(), out_dtype=torch.float32, out=residual)
        return None
    if out_dtype == torch.float32:
        return torch.mm(x, weight.t(), out_dtype=torch.float32)
    return torch.nn.functional.linear(x, weight)    # float accumulation


def linear(x, weight: torch.Tensor, out_dtype: Optional[torch.dtype] = None,
           residual: Optional[torch.Tensor] = None, gated: bool = False,
           planes_ok: bool = False, next_norm=None, activation: str = "silu", limit: Optional[float] = None):
    """x[R,K] . weight[N,K]^T, with optional neighbours.

    ``x`` is a tensor or ``NormedRows`` (a norm still to be done).  ``gated``: the weight is an
    interleaved gate/up weight and the result is act(gate) * up, ``[R, N/2]``, act being silu or what
    ``activation`` names (``GLU_ACTIVATIONS``; ``limit`` belongs to "clamped_swish").  ``residual``: the caller
    wants the product added into this float32 tensor; if the kernel in use can do that, it does and None
    is returned, otherwise the product is returned for the caller to add later, as float32 ``[R, N]`` or
    as a stack of planes ``[p, R, N]`` whose sum is meant (``add_rmsnorm`` takes either).

    ``next_norm`` = (gain, eps, dtype) with ``residual``: the caller will normalise the stream with this
    gain next; the kernel may leave that norm's operand behind, and then ``PreparedRows`` is returned
    instead of None.  ``planes_ok``: the caller also takes a plain product as float32 planes ``[p, R, N]`` whose sum, in
    order, is meant (``qk_norm_rope_write`` does).

    float32 runs the single-precision kernel.  bfloat16 accumulates in float: up to FUSED_ROWS rows on the
    weight-streaming kernel with everything folded in, up to ROWS_MAX rows (a decode step of many requests)
    on the multi-row weight-streaming kernel, more rows (prompt portions) through the library's matrix
    product, with float32 output for logits and for what goes into the stream.
    """
    dtype = x.dtype if isinstance(x, NormedRows) else x.dtype
    if dtype != weight.dtype:
        raise KernelError(f"linear: activations are {dtype} but the weight is {weight.dtype}")
    out_dtype = out_dtype or dtype
    rows, k = x.shape
    if dtype == torch.bfloat16 and weight.is_cuda and k % 8 == 0 and rows <= FUSED_ROWS \
            and (not gated or weight.shape[0] % 16 == 0):
        # Every workgroup (16 weight rows) would redo a folded norm for its own use: that pays only for
        # matrices with few rows; for the others the norm kernel runs once and the product reads its result.
        if isinstance(x, NormedRows) and not isinstance(x, PreparedRows) and weight.shape[0] > FUSED_NORM_WEIGHT_ROWS:
            # rounds where the folded norm rounds, whatever the weight's size
            x = x.prepare() if prepared_fits(rows, k) else x.materialize()
        if next_norm is not None and (residual is None or not prepared_fits(rows, weight.shape[0])
                                      or next_norm[2] != torch.bfloat16):
            next_norm = None
        return gemm_fused(x, weight, out_dtype, residual, gated, next_norm, activation=activation, limit=limit)
    x = materialize(x)
    if dtype == torch.bfloat16 and weight.is_cuda and k % 8 == 0 and rows <= ROWS_MAX \
            and (not gated or weight.shape[0] % 16 == 0):
        return gemm_rows(x, weight, out_dtype, residual, gated, may_split=planes_ok or residual is not None,
                         activation=activation, limit=limit)
    if dtype == torch.float32:
        if out_dtype != torch.float32:
            raise KernelError("linear: the float32 path produces float32")
        y = gemm_f32(x, weight)
    elif not x.is_cuda:
        raise KernelError("linear: tensor is not on the GPU")
    elif out_dtype == torch.float32 or (residual is not None and not gated):
        # float32 results for many rows, from the library's product with float output: logits, and what is
        # to be added into the float32 stream, which the kernel for few rows adds unrounded as well
        parts = inner_parts(rows, weight.shape[0], k) if residual is not None else 1
        with profile.span(profile.LIBRARY_PRODUCT, weight):
            if parts > 1:
                # [parts, rows, N]: the planes are summed, in order, by the norm kernel that adds them
                y = torch.bmm(x.view(rows, parts, k // parts).transpose(0, 1),
                              weight.view(weight.shape[0], parts, k // parts).permute(1, 2, 0), out_dtype=torch.float32)
            elif residual is not None:
                return _library_product(x, weight, torch.float32, residual)
            else:
                y = _library_product(x, weight, torch.float32, None)
    else:
        with profile.span(profile.LIBRARY_PRODUCT, weight):
            y = _library_product(x, weight, torch.bfloat16, None)
        if out_dtype != y.dtype:
            y = y.to(out_dtype)
    return swiglu(y, activation=activation, limit=limit) if gated else y


def linear_planes(x: torch.Tensor, weight: torch.Tensor, rows_of) -> list:
    """Products of several inputs ``x[planes, R, K]`` against matrices that lie one behind the other in ``weight[N, K]``
    (``rows_of`` says how many rows each has): a list of float32 ``[R, rows_of[p]]`` = x[p] . weight_p^T, which may be slices
    of one wider result.  Few bfloat16 rows against equal matrices of a multiple of 16 rows (the last may be smaller) are one
    launch; otherwise a product each, as ``linear`` would make it."""
    planes, rows, k = x.shape
    rows_of = [int(r) for r in rows_of]
    if len(rows_of) != planes or sum(rows_of) != weight.shape[0] or weight.shape[1] != k or x.dtype != weight.dtype:
        raise KernelError(f"linear_planes: inputs {tuple(x.shape)} of {x.dtype} against {tuple(weight.shape)} of {weight.dtype} in {rows_of} rows")
    starts = [sum(rows_of[:p]) for p in range(planes)]
    tiles = streamed_copy(weight) if _streamed else None
    if x.dtype == torch.bfloat16 and rows <= FUSED_ROWS and k % 8 == 0 and rows_of[0] % 16 == 0 \
            and all(r == rows_of[0] for r in rows_of[:-1]) and rows_of[-1] <= rows_of[0]:
        out = torch.empty((rows, weight.shape[0]), dtype=torch.float32, device=x.device)
        with profile.span("gemv fused", weight):
            call("leone_gemm_planes_bf16", _dev(x, "gemm x", torch.bfloat16), planes, rows_of[0],
                 _dev(weight if tiles is None else tiles, "gemm weight", torch.bfloat16), 0 if tiles is None else 1,
                 _dev(out, "gemm out"), F32, rows, weight.shape[0], k, _stream())
        return [out[:, at:at + r] for at, r in zip(starts, rows_of)]
    results = []
    for p, (at, r) in enumerate(zip(starts, rows_of)):
        part = weight[at:at + r]
        if x.dtype == torch.bfloat16 and FUSED_ROWS < rows <= ROWS_MAX and k % 8 == 0 and tiles is not None and at % 16 == 0:
            # the whole matrix's second copy is tiles of 16 rows: a part that begins at one has its own piece of it
            results.append(gemm_rows(x[p], part, torch.float32, may_split=False, tiles=tiles[at // 16:-(-(at + r) // 16)]))
        else:
            results.append(linear(x[p], part, out_dtype=torch.float32))
    return results


def argmax(logits: torch.Tensor) -> torch.Tensor:
    rows, vocab = logits.shape
    chunks = -(-vocab // library().leone_argmax_chunk())
    out = torch.empty((rows,), dtype=torch.int32, device=logits.device)
    part_value = torch.empty((rows * chunks,), dtype=torch.float32, device=logits.device)
    part_index = torch.empty((rows * chunks,), dtype=torch.int32, device=logits.device)
    call("leone_argmax", _dev(logits, "argmax logits", torch.float32), _dev(out, "argmax out"),
         _dev(part_value, "argmax partial values"), _dev(part_index, "argmax partial indices"), rows, vocab,
         _stream())
    return out


def sample_temperature(logits: torch.Tensor, temperature: torch.Tensor, uniform: torch.Tensor) -> torch.Tensor:
    """One token a row by its temperature (float64 [rows], positive) and uniform value (float64 [rows] in
    [0, 1)); -1 for a row without a finite logit."""
    rows, vocab = logits.shape
    chunks = -(-vocab // library().leone_argmax_chunk())
    out = torch.empty((rows,), dtype=torch.int32, device=logits.device)
    part_value = torch.empty((rows * chunks,), dtype=torch.float32, device=logits.device)
    part_index = torch.empty((rows * (chunks + 1),), dtype=torch.int32, device=logits.device)   # and the best of each row
    sums = torch.empty((rows * chunks,), dtype=torch.float64, device=logits.device)
    call("leone_sample_temperature", _dev(logits, "sample logits", torch.float32),
         _dev(temperature, "sample temperature", torch.float64, (rows,)),
         _dev(uniform, "sample uniform", torch.float64, (rows,)), _dev(out, "sample out"),
         _dev(part_value, "sample partial values"), _dev(part_index[:rows * chunks], "sample partial indices"),
         _dev(part_index[rows * chunks:], "sample best"), _dev(sums, "sample sums"), rows, vocab, _stream())
    return out


TOP_CANDIDATES_MAX = 256     # most candidates a row the selection kernel gives (checked against the library)


def top_candidates(logits: torch.Tensor, wanted) -> tuple:
    """The ``wanted[row]`` best finite logits of every row in the sampler's order (higher first, the lower
    id on a tie), selected on the device and brought to the host in one copy.

    Returns numpy arrays: values float32 [rows, TOP_CANDIDATES_MAX], ids int32 likewise, counts int32
    [rows]; row r is filled up to counts[r] (fewer than it wanted only if it has fewer finite logits)."""
    if library().leone_top_candidates_max() != TOP_CANDIDATES_MAX:
        raise KernelError("the kernel library was built for another number of candidates")
    rows, vocab = logits.shape
    wanted = [int(k) for k in wanted]
    if len(wanted) != rows or not all(1 <= k <= TOP_CANDIDATES_MAX for k in wanted):
        raise KernelError(f"top_candidates: one count in 1..{TOP_CANDIDATES_MAX} for each of {rows} rows, found {wanted}")
    room = rows * TOP_CANDIDATES_MAX
    flat = torch.empty((rows + 2 * room,), dtype=torch.int32, device=logits.device)   # counts | values | ids
    # The kernel selects the largest count for every row, best first: a row that wants fewer takes the first.
    call("leone_top_candidates", _dev(logits, "candidate logits", torch.float32),
         _dev(flat[rows:rows + room], "candidate values"), _dev(flat[rows + room:], "candidate ids"),
         _dev(flat[:rows], "candidate counts"), rows, vocab, max(wanted), _stream())
    host = flat.cpu().numpy()
    counts = np.where(host[:rows] < 0, -1, np.minimum(host[:rows], np.asarray(wanted, dtype=np.int32)))
    return (host[rows:rows + room].view("float32").reshape(rows, TOP_CANDIDATES_MAX),
            host[rows + room:].reshape(rows, TOP_CANDIDATES_MAX), counts)


TRUNCATED_STAGES = 8         # most truncation stages of a row that is drawn on the device (checked against the library)
TRUNCATION_KINDS = {"top_k": 0, "top_p": 1, "min_p": 2}


def truncated_draw_supported(stages) -> bool:
    """Whether ``sample_truncated`` serves a row with these (stage, value) pairs: top-k first with k at most
    TOP_CANDIDATES_MAX, then top-k, top-p and min-p in any order, TRUNCATED_STAGES at most in all."""
    stages = list(stages)
    return (0 < len(stages) <= TRUNCATED_STAGES and all(name in TRUNCATION_KINDS for name, _ in stages)
            and stages[0][0] == "top_k" and 1 <= int(stages[0][1]) <= TOP_CANDIDATES_MAX)


def truncated_rows(draws) -> np.ndarray:
    """The parameters of ``sample_truncated`` as a host array, float64 [rows, 3 + 2 * TRUNCATED_STAGES]: ``draws``
    holds for each row either None (the row is skipped and gets -1) or (temperature, uniform value,
    [(stage, value), ...]) with stages that ``truncated_draw_supported`` accepts."""
    lib = library()
    if (lib.leone_sample_truncated_stages() != TRUNCATED_STAGES or lib.leone_top_candidates_max() != TOP_CANDIDATES_MAX
            or lib.leone_sample_truncated_params() != 3 + 2 * TRUNCATED_STAGES):
        raise KernelError("the kernel library was built for another table of truncation stages")
    draws = list(draws)
    table = np.zeros((len(draws), 3 + 2 * TRUNCATED_STAGES), dtype=np.float64)
    for r, draw in enumerate(draws):
        if draw is None:
            continue
        temperature, uniform, stages = draw
        stages = list(stages)
        if not truncated_draw_supported(stages):
            raise KernelError(f"sample_truncated: row {r}: stages {stages} are not drawn on the device")
        if not (math.isfinite(temperature) and temperature > 0.0 and 0.0 <= uniform < 1.0):
            raise KernelError(f"sample_truncated: row {r}: temperature {temperature} or uniform value {uniform} out of range")
        for name, value in stages:
            if name == "top_k" and not (value >= 1 and int(value) == value) or name != "top_k" and not 0.0 < value <= 1.0:
                raise KernelError(f"sample_truncated: row {r}: {name} {value} out of range")
        table[r, 0], table[r, 1], table[r, 2] = temperature, uniform, len(stages)
        for s, (name, value) in enumerate(stages):
            # top-k beyond every vocabulary keeps everything: the value only has to stay a number the kernel can compare
            table[r, 3 + 2 * s], table[r, 4 + 2 * s] = TRUNCATION_KINDS[name], min(float(value), 2.0 ** 31)
    return table


def truncated_table(draws, device) -> torch.Tensor:
    """``truncated_rows`` on the device."""
    return torch.from_numpy(truncated_rows(draws)).to(device)


def sample_truncated(logits: torch.Tensor, draws) -> torch.Tensor:
    """One token a row (int32 on the device) by temperature sampling with truncation stages, top-k first:
    selection, stages and draw in one launch, nothing comes to the host.  ``draws``: what ``truncated_table``
    takes, or the table it made (float64 on the device).  -1 for a skipped row and for a row without a finite
    logit."""
    rows, vocab = logits.shape
    params = draws if isinstance(draws, torch.Tensor) else truncated_table(draws, logits.device)
    if params.shape != (rows, 3 + 2 * TRUNCATED_STAGES):
        raise KernelError(f"sample_truncated: {rows} rows of logits, a table of {tuple(params.shape)}")
    out = torch.empty((rows,), dtype=torch.int32, device=logits.device)
    call("leone_sample_truncated", _dev(logits, "sample logits", torch.float32),
         _dev(params, "sample stages", torch.float64), _dev(out, "sample out"), rows, vocab, _stream())
    return out


__all__ = [name for name in dir() if not name.startswith("_")]


# ---- layers that keep state of their own per request ---------------------------------------------------------
ACTIVATIONS = {None: 0, "none": 0, "sigmoid": 1, "silu": 2}


class NormedDelta:
    """What a sublayer adds to the stream, still to be normalised: ``norm`` (a norm part) is applied to
    ``rows`` (float32 ``[rows, hidden]``) before the sum.  The norm part that runs next takes it in place of a
    delta and does both in one pass (``add_layernorm``); any other consumer asks for ``materialize()``."""

    def __init__(self, rows: torch.Tensor, norm):
        self.rows, self.norm = rows, norm

    def materialize(self) -> torch.Tensor:
        return self.norm.apply(self.rows)


def add_layernorm(x: torch.Tensor, delta: Optional[torch.Tensor], gain: Optional[torch.Tensor],
                  bias: Optional[torch.Tensor], eps: float, out_dtype: Optional[torch.dtype],
                  rows: Optional[torch.Tensor] = None, delta_norm: Optional[tuple] = None,
                  conv: Optional[tuple] = None) -> Optional[torch.Tensor]:
    """x += delta, where ``delta_norm`` = (gain, bias, eps) says that the delta goes through a layer norm of its
    own first; then y = (x - mean) / sqrt(var + eps) * gain + bias in ``out_dtype`` (None: no y, only the sum).
    With ``rows`` y[i] comes from row rows[i] and x is not written.  Means and variances are float.
    ``conv`` = (weight ``[hidden, taps]``, state, step, write_state), for a step of single rows only: what comes
    out is y + conv(y) as ``causal_conv(add_input=True)`` gives it, and the state has moved on, in the same launch."""
    n, hidden = x.shape
    n_out = n if rows is None else rows.numel()
    if delta is not None and delta.dtype != torch.float32:
        delta = delta.float()
    y = torch.empty((n_out, hidden), dtype=out_dtype, device=x.device) if out_dtype is not None else None
    vectors = [v for v in (gain, bias) + tuple(delta_norm[:2] if delta_norm else ()) if v is not None]
    if len({v.dtype for v in vectors}) > 1:
        raise KernelError("add_layernorm: gains and biases must share one type")
    call("leone_add_layernorm", _dev(x, "stream", torch.float32), _dev(delta, "delta", torch.float32, (n, hidden)),
         _dev(delta_norm[0], "delta gain", None, (hidden,)) if delta_norm else 0,
         _dev(delta_norm[1], "delta bias", None, (hidden,)) if delta_norm else 0,
         float(delta_norm[2]) if delta_norm else 0.0,
         _dev(gain, "gain", None, (hidden,)), _dev(bias, "bias", None, (hidden,)),
         _code(vectors[0], "gain") if vectors else F32, float(eps), _dev(y, "normed rows"),
         _CODES[out_dtype] if out_dtype is not None else F32,
         _dev(rows, "rows", torch.int32) if rows is not None else 0, n_out, hidden, *_folded_conv(conv, n, hidden), _stream())
    return y


def _folded_conv(conv, rows: int, hidden: int) -> tuple:
    """The arguments of a convolution folded into ``add_layernorm``."""
    if conv is None:
        return 0, F32, 0, 0, 0, 0, 0, 0
    weight, state, step, write_state = conv
    taps = weight.shape[1]
    if not step.decode_only or step.rows != rows:
        raise KernelError("add_layernorm: a convolution is folded in only for a step of single rows")
    if tuple(weight.shape) != (hidden, taps) or state.dtype != torch.float32 or tuple(state.shape[1:]) != (taps - 1, hidden):
        raise KernelError(f"add_layernorm: conv weight {tuple(weight.shape)} and state {tuple(state.shape)} do not fit rows of {hidden}")
    return (_dev(weight, "conv weight"), _code(weight, "conv weight"), taps, _dev(state, "conv state"), 1 if write_state else 0,
            _dev(step.positions, "positions", torch.int32, (rows,)), _dev(step.row_entry, "row map", torch.int32, (rows,)),
            _dev(step.entry_slots, "slots", torch.int32))


def entry_spans(step) -> torch.Tensor:
    """int32 ``[entries, 4]`` on the device: first row and end of every entry's rows in the step, the state slot
    it reads (-1 at a sequence's start: it starts from zeros) and the slot it writes; made once a step from
    the row -> entry map (so that it is there too when a step is replayed from a recording)."""
    spans = getattr(step, "spans", None)
    if spans is None:
        entries = step.entry_slots.numel()
        spans = torch.empty((entries, 4), dtype=torch.int32, device=step.row_entry.device)
        call("leone_entry_spans", _dev(step.row_entry, "row map", torch.int32, (step.rows,)),
             _dev(step.positions, "positions", torch.int32, (step.rows,)), _dev(step.entry_slots, "slots", torch.int32),
             step.rows, _dev(spans, "spans"), _stream())
        step.spans = spans
    return spans


# Rows of a chunk when a long portion's recurrence is walked chunk by chunk, side by side, and the portions that
# are (at least so many rows): (chunk, from).  The outer-product recurrences chain their chunks by a factor, the
# delta rule by a matrix product a chunk, so its chunks are longer.
OUTER_CHUNKS = (64, 256)
DELTA_CHUNKS = (256, 512)


def chunk_plan(step, chunk: int, chunked_from: int):
    """How the recurrences of a step with long portions are walked (``outer_scan``): None if the step has none (or
    is replayed from a recording: then the host does not know its entries).  Else int32 tables on the device:
    ``chunks`` ``[c, 4]`` (first row, end, -1, chunk index) of the long portions' chunks, ``again`` the same chunks
    reading (chunk index, -1), ``links`` ``[l, 4]`` (state slot, whether the sequence starts here, first chunk, end)
    one a long portion, and ``short`` ``[s, 4]`` the other entries as single segments from and into their slots."""
    plans = step.plan if isinstance(step.plan, dict) else {}
    step.plan = plans
    key = (chunk, chunked_from)
    if key in plans:
        return plans[key]
    plans[key] = None
    if not any(e.count >= chunked_from for e in step.entries):
        return None
    chunks, again, links, short = [], [], [], []
    for e in step.entries:
        if e.count >= chunked_from:
            first_chunk = len(chunks)
            for at in range(0, e.count, chunk):
                rows = (e.first_row + at, e.first_row + min(at + chunk, e.count))
                again.append(rows + (len(chunks), -1))
                chunks.append(rows + (-1, len(chunks)))
            links.append((e.slot, 1 if e.start == 0 else 0, first_chunk, len(chunks)))
        else:
            short.append((e.first_row, e.first_row + e.count, -1 if e.start == 0 else e.slot, e.slot))
    flat = torch.tensor(chunks + again + links + short, dtype=torch.int32).to(step.device)
    c, l = len(chunks), len(links)
    plans[key] = {"chunks": flat[:c], "again": flat[c:2 * c], "links": flat[2 * c:2 * c + l], "short": flat[2 * c + l:]}
    return plans[key]


def causal_conv(x: torch.Tensor, weight: torch.Tensor, state: torch.Tensor, step, out_dtype: torch.dtype,
                add_input: bool = False, activation: Optional[str] = None, write_state: bool = True,
                bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """out[t, c] = (x[t, c] if ``add_input``) + sum_j weight[c, j] * x[t - (taps - 1) + j, c] (+ ``bias[c]``), then
    the activation; rows before a portion come from ``state`` (float32 ``[slots, taps - 1, channels]``: a request's
    last inputs), zeros before position 0.  ``x`` may be a column slice of wider rows.  Leaves the state
    brought up to date unless told not to.  ``bias`` ``[channels]`` comes in the filters' type."""
    rows, channels = x.shape
    taps = weight.shape[1]
    if tuple(weight.shape) != (channels, taps) or x.dim() != 2 or x.stride(1) != 1:
        raise KernelError(f"causal_conv: weight {tuple(weight.shape)} for rows of {channels} channels")
    if state.dtype != torch.float32 or tuple(state.shape[1:]) != (taps - 1, channels):
        raise KernelError(f"causal_conv: state {tuple(state.shape)} is not [slots, {taps - 1}, {channels}] float32")
    if not x.is_cuda:
        raise KernelError("causal_conv: tensor is not on the GPU")
    if bias is not None and bias.dtype != weight.dtype:
        raise KernelError(f"causal_conv: a bias of {bias.dtype} beside filters of {weight.dtype}")
    out = torch.empty((rows, channels), dtype=out_dtype, device=x.device)
    spans = entry_spans(step)
    single_rows = bool(step.decode_only) and step.entry_slots.numel() == rows
    call("leone_causal_conv_biased", x.data_ptr(), _code(x, "conv input"), x.stride(0), _dev(out, "conv out"), _CODES[out_dtype],
         channels, _dev(weight, "conv weight"), _dev(bias, "conv bias", None, (channels,)), _code(weight, "conv weight"),
         _dev(state, "conv state"),
         1 if write_state else 0, _dev(spans, "spans"), spans.shape[0],
         _dev(step.positions, "positions", torch.int32, (rows,)), _dev(step.row_entry, "row map", torch.int32, (rows,)),
         _dev(step.entry_slots, "slots", torch.int32), rows, channels, taps, 1 if add_input else 0,
         ACTIVATIONS[activation], 1 if single_rows else 0, _stream())
    return out


def head_norm_gate(o: torch.Tensor, heads: int, vdim: int, eps: float, out_dtype: torch.dtype,
                   gain: Optional[torch.Tensor] = None, gate: Optional[torch.Tensor] = None,
                   activation: Optional[str] = None, denominator: Optional[tuple] = None,
                   gate_first: bool = False) -> torch.Tensor:
    """Head by head: o (float32 ``[rows, heads * vdim]``), divided by max(|dot|, exp(-top)) + 1e-6 if
    ``denominator`` = (dot, top) (float32 ``[rows, heads]``) comes, over its root mean square, times ``gain``
    (``[heads * vdim]``, or ``[vdim]`` shared by the heads), times activation(gate) (float32 rows of heads * vdim,
    possibly a slice of wider rows).  ``gate_first``: the gate multiplies ahead of the norm, so the root mean square
    is that of the gated values.  A "head" is whatever run of ``vdim`` columns is normed by itself."""
    rows = o.shape[0]
    out = torch.empty((rows, heads * vdim), dtype=out_dtype, device=o.device)
    per_head = 0
    if gain is not None:
        if gain.numel() == heads * vdim and heads > 1:
            per_head = 1
        elif gain.numel() != vdim:
            raise KernelError(f"head_norm_gate: a gain of {gain.numel()} for {heads} heads of {vdim}")
    gate_at, gate_stride = _strided_rows(gate, "head_norm_gate gate", rows, heads * vdim)
    dot, top = denominator if denominator is not None else (None, None)
    call("leone_head_norm_gate_ordered", _dev(o, "read-outs", torch.float32, (rows, heads * vdim)),
         _dev(dot, "dot", torch.float32, (rows, heads)), _dev(top, "top", torch.float32, (rows, heads)),
         _dev(gain, "gain"), _code(gain, "gain") if gain is not None else F32, per_head, gate_at, gate_stride,
         ACTIVATIONS[activation], 1 if gate_first else 0, float(eps), _dev(out, "out"), _CODES[out_dtype], rows, heads, vdim, _stream())
    return out


def rms_mix(branches, gains, eps: float, scale: float) -> torch.Tensor:
    """scale * sum_b rms(branches[b]) * gains[b]: every branch (float32 ``[rows, hidden]``) over its root mean
    square along the row, times its gain."""
    rows, hidden = branches[0].shape
    if len(branches) != len(gains) or len({g.dtype for g in gains}) != 1:
        raise KernelError("rms_mix: one gain a branch, all of one type")
    out = torch.empty((rows, hidden), dtype=torch.float32, device=branches[0].device)
    row_ptrs = (ctypes.c_void_p * len(branches))(*[_dev(b, "branch", torch.float32, (rows, hidden)) for b in branches])
    gain_ptrs = (ctypes.c_void_p * len(gains))(*[_dev(g, "branch gain", None, (hidden,)) for g in gains])
    call("leone_rms_mix", ctypes.cast(row_ptrs, ctypes.c_void_p), ctypes.cast(gain_ptrs, ctypes.c_void_p),
         _code(gains[0], "branch gain"), len(branches), float(eps), float(scale), _dev(out, "out"), rows, hidden, _stream())
    return out


def weighted_mix(branches, weights) -> torch.Tensor:
    """sum_b weights[b] * branches[b]: float32 tensors of one shape, 1 to 4 of them, nothing normed."""
    shape = tuple(branches[0].shape)
    if len(branches) != len(weights) or not 1 <= len(branches) <= 4:
        raise KernelError("weighted_mix: one weight for each of 1 to 4 branches")
    out = torch.empty(shape, dtype=torch.float32, device=branches[0].device)
    row_ptrs = (ctypes.c_void_p * len(branches))(*[_dev(b, "branch", torch.float32, shape) for b in branches])
    factors = (ctypes.c_float * len(weights))(*[float(w) for w in weights])
    call("leone_weighted_mix", ctypes.cast(row_ptrs, ctypes.c_void_p), ctypes.cast(factors, ctypes.c_void_p), len(branches),
         _dev(out, "out"), out.numel(), _stream())
    return out


def bias_span_norm(rows: torch.Tensor, bias: Optional[torch.Tensor], spans, eps: float, round_to: Optional[torch.dtype] = None) -> torch.Tensor:
    """In place on float32 ``rows`` ``[n, width]``: the first ``len(bias)`` columns get their bias (None: none) and, with
    ``round_to`` bfloat16, that type's rounding (what a product kept in the engine's type would hold); then every span
    ``(offset, width, gain)`` is divided by its root mean square over the whole span, eps inside the root, and multiplied
    by ``gain`` ``[width]``.  A span may name a fourth value, the number of elements its mean is taken over (a span
    that holds columns of zeros that do not count).  Up to four spans that do not overlap."""
    n, width = rows.shape
    spans = [tuple(span) + ((span[1],) if len(span) == 3 else ()) for span in spans]
    counts = (ctypes.c_int * max(len(spans), 1))(*[int(c) for _, _, _, c in spans])
    spans = [span[:3] for span in spans]
    gains = [g for _, _, g in spans]
    if len({g.dtype for g in gains}) > 1:
        raise KernelError("bias_span_norm: the gains must come in one type")
    biased = bias.numel() if bias is not None else (width if round_to == torch.bfloat16 else 0)
    offsets = (ctypes.c_int * max(len(spans), 1))(*[int(o) for o, _, _ in spans])
    widths = (ctypes.c_int * max(len(spans), 1))(*[int(w) for _, w, _ in spans])
    gain_ptrs = (ctypes.c_void_p * max(len(spans), 1))(*[_dev(g, "span gain", None, (int(w),)) for _, w, g in spans])
    call("leone_bias_span_norm", _dev(rows, "rows", torch.float32), width, n, _dev(bias, "bias"),
         _code(bias, "bias") if bias is not None else F32, biased, 1 if round_to == torch.bfloat16 else 0,
         ctypes.cast(offsets, ctypes.c_void_p), ctypes.cast(widths, ctypes.c_void_p), ctypes.cast(counts, ctypes.c_void_p),
         ctypes.cast(gain_ptrs, ctypes.c_void_p), _code(gains[0], "span gain") if gains else F32, len(spans), float(eps), _stream())
    return rows


def bias_glu(gate_up: torch.Tensor, bias: Optional[torch.Tensor], out_dtype: torch.dtype, activation: str = "silu") -> torch.Tensor:
    """act(gate + b_gate) * (up + b_up) from rows ``[gate | up]`` ``[n, 2 ff]`` (one half behind the other) and a bias of
    the same order ``[2 ff]`` (None: none) -> ``[n, ff]`` in ``out_dtype``."""
    n, both = gate_up.shape
    if both % 2:
        raise KernelError(f"bias_glu: rows of {both} are no [gate | up]")
    out = torch.empty((n, both // 2), dtype=out_dtype, device=gate_up.device)
    call("leone_bias_glu", _dev(gate_up, "gate and up"), _code(gate_up, "gate and up"), _dev(bias, "bias", None, (both,)),
         _code(bias, "bias") if bias is not None else F32, _dev(out, "out"), _CODES[out_dtype], n, both // 2,
         _gate_code(activation), _stream())
    return out


def add_bias(x: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """x[r, c] += bias[c], in place on float32 rows."""
    n, width = x.shape
    call("leone_add_bias", _dev(x, "rows", torch.float32), _dev(bias, "bias", None, (width,)), _code(bias, "bias"), n, width, _stream())
    return x


def relu_squared(x: torch.Tensor) -> torch.Tensor:
    """max(x, 0)^2."""
    out = torch.empty_like(x)
    call("leone_relu_squared", _dev(x, "values"), _dev(out, "out"), _code(x, "values"), x.numel(), _stream())
    return out


def head_gate(out: torch.Tensor, gate: torch.Tensor, heads: int, vdim: int) -> torch.Tensor:
    """out[r, h, :] *= sigmoid(gate[r, h]) in place; ``gate`` float32, possibly a slice of wider rows."""
    rows = out.shape[0]
    gate_at, gate_stride = _strided_rows(gate, "head gate", rows, heads)
    call("leone_head_gate", _dev(out, "values", None, (rows, heads * vdim)), _code(out, "values"), gate_at, gate_stride,
         rows, heads, vdim, _stream())
    return out


def scan_max_dim() -> int:
    return int(library().leone_scan_max_dim())


MEMORY_CHUNKS_FROM = 32     # portions of at least so many rows go through a memory with one decay a head as ``chunked_memory``


def chunked_memory_supported(dim: int) -> bool:
    return dim <= library().leone_chunk_max_dim()


def chunked_memory(rows: torch.Tensor, columns: dict, plan: dict, state: torch.Tensor, out: torch.Tensor, heads: int, kv_heads: int,
                   dim: int, vdim: int, *, q_scale: float, k_scale: float, activation: Optional[str] = None,
                   decay: Optional[torch.Tensor] = None, delta: Optional[tuple] = None, write_state: bool = True) -> None:
    """The long portions of a step (``plan``: ``chunk_plan`` with chunks of ``leone_chunk_rows()`` rows) through a matrix memory
    with one decay a head, chunk by chunk on the matrix cores in float: S <- g S + k u^T, o = S^T q, with ``decay`` (float32
    ``[heads]``) and u = v, or the delta rule's u = beta (v - g S^T k): ``delta`` = (strengths' pre-activations ``[rows, >=
    heads]``, step sizes' pre-activations likewise, rate_log and step_bias ``[heads]``, unit_eps).  Fills the portions' rows of
    ``out`` and moves their states."""
    chunks, links = plan["chunks"], plan["links"]
    n, count = rows.shape[0], chunks.shape[0]
    size = library().leone_chunk_workspace(dim, vdim, 1 if delta is not None else 0)
    workspace = torch.empty((count * heads * size,), dtype=torch.float32, device=rows.device)
    beta, step_size, rate_log, step_bias, unit_eps = delta if delta is not None else (None, None, None, None, 0.0)
    beta_at, beta_stride = _strided_rows(beta, "write strengths", n, heads)
    step_at, step_stride = _strided_rows(step_size, "step sizes", n, heads)
    call("leone_chunked_memory", _dev(rows, "q, k, v", torch.float32), rows.shape[1], columns["q"], columns["k"], columns["v"],
         1 if activation == "silu" else 0, float(q_scale), float(k_scale), float(unit_eps), beta_at, beta_stride, step_at, step_stride,
         _dev(rate_log, "rate", None, (heads,)), _dev(step_bias, "step bias", None, (heads,)),
         _code(rate_log, "rate") if rate_log is not None else F32,
         _dev(decay, "decay", torch.float32, (heads,)) if delta is None else 0, _dev(chunks, "chunks", torch.int32), count,
         _dev(links, "links", torch.int32), links.shape[0], _dev(workspace, "workspace"), _dev(state, "state", torch.float32),
         state.stride(0), 1 if write_state else 0, _dev(out, "out", torch.float32, (n, heads * vdim)), heads, kv_heads, dim, vdim, _stream())


def outer_scan(proj: torch.Tensor, columns: dict, state: torch.Tensor, step, heads: int, dim: int, vdim: int, *,
               gates: Optional[dict] = None, decay: Optional[torch.Tensor] = None, q_scale: float = 1.0,
               k_scale: float = 1.0, cos: Optional[torch.Tensor] = None, sin: Optional[torch.Tensor] = None,
               activation: Optional[str] = None, write_state: bool = True):
    """The matrix-memory recurrence S_t = a_t S_(t-1) + b_t k_t v_t^T, o_t = S_t^T q_t over every entry's rows,
    from and into ``state`` (float32 ``[slots, heads, dim * vdim]``, with ``gates`` ``dim * vdim + dim + 1``: the
    normaliser and the running maximum ride along).  ``proj`` is float32 ``[rows, width]``; ``columns`` names the
    first column of q, k and v (and, with ``gates``, of the input and forget gates' pre-activations "i", "f").
    ``gates`` = {"i_bias", "f_bias", "cap"}: exponential gates with a running maximum that starts at 0; else
    ``decay`` (float32 ``[heads]``) with b = 1.  ``cos``/``sin``: rotary tables for q and k.  ``activation`` "silu": q, k and v
    pass through it first.
    Returns o float32 ``[rows, heads * vdim]`` and, with gates, (dot, top) for ``head_norm_gate``.

    Single tokens and short portions are walked row by row.  A long portion (``OUTER_CHUNKS``) is cut into chunks
    that are walked side by side: every chunk from zeros, the chunks' end states chained, every chunk once more
    from the state it starts with."""
    rows, width = proj.shape
    per_head = dim * vdim + (dim + 1 if gates else 0)
    if state.dtype != torch.float32 or state.dim() != 3 or tuple(state.shape[1:]) != (heads, per_head) or not state.is_contiguous():
        raise KernelError(f"outer_scan: state {tuple(state.shape)} is not [slots, {heads}, {per_head}] float32")
    if activation not in (None, "silu"):
        raise KernelError(f"outer_scan: q, k and v pass as they are or through silu, not {activation!r}")
    spans = entry_spans(step)
    device = proj.device
    out = torch.empty((rows, heads * vdim), dtype=torch.float32, device=device)
    dot = top = coef = None
    if gates:
        dot = torch.empty((rows, heads), dtype=torch.float32, device=device)
        top = torch.empty((rows, heads), dtype=torch.float32, device=device)
        coef = torch.empty((rows, heads, 2), dtype=torch.float32, device=device)
        if gates["i_bias"].dtype != gates["f_bias"].dtype:
            raise KernelError("outer_scan: the gates' biases must share one type")
        call("leone_exp_gates", _dev(proj, "projection", torch.float32), width, columns["i"], columns["f"],
             _dev(gates["i_bias"], "i bias", None, (heads,)), _dev(gates["f_bias"], "f bias", None, (heads,)),
             _code(gates["i_bias"], "i bias"), float(gates["cap"]), _dev(spans, "spans"), spans.shape[0],
             _dev(state, "state"), state.stride(0), per_head, dim * vdim + dim, 1 if write_state else 0,
             _dev(coef, "coefficients"), _dev(top, "top"), heads, _stream())
    rotary_dim = 2 * cos.shape[1] if cos is not None else 0

    def walk(segments, state_in, state_out, no_input=False, accumulate=False, product=None):
        call("leone_outer_scan", _dev(proj, "projection", torch.float32), width, columns["q"], columns["k"], columns["v"],
             _dev(coef, "coefficients"), _dev(decay, "decay", torch.float32, (heads,)) if decay is not None else 0,
             1 if no_input else 0, 1 if accumulate else 0, 1 if gates else 0, float(q_scale), float(k_scale),
             1 if activation == "silu" else 0,
             _dev(cos, "rope cos", torch.float32), _dev(sin, "rope sin", torch.float32), rotary_dim,
             cos.shape[0] if cos is not None else 0, _dev(step.positions, "positions", torch.int32, (rows,)),
             _dev(segments, "segments", torch.int32), segments.shape[0],
             _dev(state_in, "state read"), state_in.stride(0) if state_in is not None else 0,
             _dev(state_out, "state written"), state_out.stride(0) if state_out is not None else 0, per_head,
             _dev(product, "decay products"), _dev(out, "out"), _dev(dot, "dot"), heads, dim, vdim, _stream())

    plan = None
    if not gates and cos is None and chunked_memory_supported(dim):
        plan = chunk_plan(step, library().leone_chunk_rows(), MEMORY_CHUNKS_FROM)
        if plan is not None:
            chunked_memory(proj, columns, plan, state, out, heads, heads, dim, vdim, q_scale=q_scale, k_scale=k_scale,
                           activation=activation, decay=decay, write_state=write_state)
            if plan["short"].shape[0]:
                walk(plan["short"], state, state if write_state else None)
            return out, None
    else:
        plan = chunk_plan(step, *OUTER_CHUNKS)
    if plan is None:
        walk(spans, state, state if write_state else None)
    else:
        chunks = plan["chunks"]
        work = torch.empty((chunks.shape[0], heads, per_head), dtype=torch.float32, device=device)
        product = torch.empty((chunks.shape[0], heads), dtype=torch.float32, device=device)
        walk(chunks, None, work, product=product)
        call("leone_outer_chain", _dev(plan["links"], "links", torch.int32), plan["links"].shape[0], _dev(work, "work"),
             work.stride(0), _dev(product, "decay products"), _dev(state, "state"), state.stride(0), per_head,
             dim * vdim + (dim if gates else 0), heads, 1 if write_state else 0, _stream())
        walk(plan["again"], work, None, no_input=True, accumulate=True)
        if plan["short"].shape[0]:
            walk(plan["short"], state, state if write_state else None)
    return (out, (dot, top)) if gates else (out, None)


def delta_scan(qkv: torch.Tensor, columns: dict, beta: torch.Tensor, step_size: torch.Tensor, rate_log: torch.Tensor,
               step_bias: torch.Tensor, state: torch.Tensor, step, heads: int, kv_heads: int, dim: int, vdim: int,
               q_scale: float, unit_eps: float, write_state: bool = True) -> torch.Tensor:
    """The gated delta rule over every entry's rows: S <- g * S with g = exp(-exp(rate_log) * softplus(step_size +
    step_bias)) per head and key channel, u = sigmoid(beta) (v - S^T k), S <- S + k u^T, o = S^T q, with q and k
    made unit vectors per head (x / sqrt(sum x^2 + unit_eps)) and q times ``q_scale``.  With a ``step_bias`` of one value a head
    there is one step size, and so one decay, a head (``step_size`` ``[rows, heads]``).  ``qkv`` float32 rows
    holding q and k (``kv_heads`` heads of ``dim``) and v (``heads`` of ``vdim``) at ``columns``; ``beta`` float32
    ``[rows, heads]`` and ``step_size`` ``[rows, heads * dim]`` may be slices of wider rows.  ``state`` float32
    ``[slots, heads, dim, vdim]``.  Returns o float32 ``[rows, heads * vdim]``.

    Long portions are walked in chunks side by side, as in ``outer_scan``; what a chunk's rows do to a state that
    comes in is no mere factor here but a matrix ``[dim, dim]``, which the first walk finds by carrying the unit
    vectors along as further columns."""
    rows = qkv.shape[0]
    if state.dtype != torch.float32 or tuple(state.shape[1:]) != (heads, dim, vdim) or not state.is_contiguous():
        raise KernelError(f"delta_scan: state {tuple(state.shape)} is not [slots, {heads}, {dim}, {vdim}] float32")
    if rate_log.dtype != step_bias.dtype:
        raise KernelError("delta_scan: rate and step bias must share one type")
    spans = entry_spans(step)
    device = qkv.device
    out = torch.empty((rows, heads * vdim), dtype=torch.float32, device=device)
    beta_at, beta_stride = _strided_rows(beta, "delta_scan beta", rows, heads)
    per_head = step_bias.numel() == heads and dim > 1
    step_at, step_stride = _strided_rows(step_size, "delta_scan step", rows, heads if per_head else heads * dim)

    def walk(segments, state_in, state_out, no_input=False, accumulate=False, transition=None):
        call("leone_delta_scan", _dev(qkv, "q, k, v", torch.float32), qkv.shape[1], columns["q"], columns["k"], columns["v"],
             beta_at, beta_stride, step_at, step_stride, 1 if per_head else 0, _dev(rate_log, "rate", None, (heads,)),
             _dev(step_bias, "step bias", None, (heads if per_head else heads * dim,)), _code(rate_log, "rate"), float(q_scale), float(unit_eps),
             1 if no_input else 0, 1 if accumulate else 0, _dev(segments, "segments", torch.int32), segments.shape[0],
             _dev(state_in, "state read"), state_in.stride(0) if state_in is not None else 0,
             _dev(state_out, "state written"), state_out.stride(0) if state_out is not None else 0,
             _dev(transition, "transitions"), _dev(out, "out"), heads, kv_heads, dim, vdim, _stream())

    plan = None
    if per_head and chunked_memory_supported(dim):
        plan = chunk_plan(step, library().leone_chunk_rows(), MEMORY_CHUNKS_FROM)
        if plan is not None:
            chunked_memory(qkv, columns, plan, state, out, heads, kv_heads, dim, vdim, q_scale=q_scale, k_scale=1.0,
                           delta=(beta, step_size, rate_log, step_bias, unit_eps), write_state=write_state)
            if plan["short"].shape[0]:
                walk(plan["short"], state, state if write_state else None)
            return out
    else:
        plan = chunk_plan(step, *DELTA_CHUNKS)
    if plan is None:
        walk(spans, state, state if write_state else None)
    else:
        chunks = plan["chunks"]
        work = torch.empty((chunks.shape[0], heads, dim, vdim), dtype=torch.float32, device=device)
        transition = torch.empty((chunks.shape[0], heads, dim, dim), dtype=torch.float32, device=device)
        walk(chunks, None, work, transition=transition)
        call("leone_delta_chain", _dev(plan["links"], "links", torch.int32), plan["links"].shape[0], _dev(work, "work"),
             work.stride(0), _dev(transition, "transitions"), _dev(state, "state"), state.stride(0), heads, dim, vdim,
             1 if write_state else 0, _stream())
        walk(plan["again"], work, None, no_input=True, accumulate=True)
        if plan["short"].shape[0]:
            walk(plan["short"], state, state if write_state else None)
    return out


# ---- a norm behind the sublayer, routed experts ----------------------------------------------------------------
def add_normed(x: torch.Tensor, delta: Optional[torch.Tensor], gain: Optional[torch.Tensor], eps: float,
               out_dtype: Optional[torch.dtype] = None, then: Optional[tuple] = None,
               rows: Optional[torch.Tensor] = None) -> Optional[torch.Tensor]:
    """x += rmsnorm(delta) * gain in the float32 stream (``delta`` float32 ``[n, hidden]`` or planes ``[p, n, hidden]``
    whose sum, in order, is meant; None: nothing is added).  What comes back: with ``out_dtype`` the new rows of
    the stream in that type (what the next sublayer's products read); with ``then = (gain2, eps2, dtype)`` instead
    rmsnorm(x) * gain2 of the new rows, of the rows ``rows`` (int32 indices) only if given, and then the stream
    itself is left as it was."""
    n, hidden = x.shape
    if delta is not None and delta.dtype != torch.float32:
        delta = delta.float()
    stacked = delta is not None and delta.dim() == 3
    planes = delta.shape[0] if stacked else 1
    if rows is not None and then is None:
        raise KernelError("add_normed: picked rows come with a second norm")
    n_out = n if rows is None else rows.numel()
    kind = then[2] if then is not None else out_dtype
    if delta is None and kind is None:
        return None
    if delta is None and then is None and kind == torch.float32:
        return x                                   # nothing to add, nothing to convert
    same = then is None and kind == torch.float32          # the stream itself is what the next products read
    y = torch.empty((n_out, hidden), dtype=kind, device=x.device) if (kind is not None and not same) else None
    call("leone_add_normed", _dev(x, "stream", torch.float32),
         _dev(delta, "delta", torch.float32, (planes, n, hidden) if stacked else (n, hidden)), planes, n * hidden,
         _dev(gain, "gain", None, (hidden,)) if delta is not None else 0,
         _code(gain, "gain") if delta is not None else F32, float(eps),
         _dev(y, "rows out"), _CODES[kind] if kind is not None else F32,
         _dev(then[0], "second gain", None, (hidden,)) if then is not None else 0,
         _code(then[0], "second gain") if then is not None else F32, float(then[1]) if then is not None else 0.0,
         _dev(rows, "rows", torch.int32) if rows is not None else 0, n_out, hidden, _stream())
    return x if same else y


ROUTER_SCORES = {"softmax": 0, "sigmoid": 1}     # how a router turns its logits into scores
# what experts put on gate and up: a gate activation, or "clamped_swish" (gate and up held to a limit, see ``glu_value``)
EXPERT_ACTIVATIONS = GLU_ACTIVATIONS                               # of experts with a gate
PLAIN_ACTIVATIONS = {**GATE_ACTIVATIONS, "relu2": 3}                # of experts without one


class RouterRule:
    """How a router scores and weighs (the defaults are a softmax router whose winners' scores are renormalised):
    ``score`` "softmax" over all outputs or "sigmoid" of each; ``group_best``: a group's score is the sum of its so
    many best choice scores; ``renormalize``: the winners' scores over their sum, else the scores themselves;
    ``scale`` multiplies the weights."""

    def __init__(self, score: str = "softmax", group_best: int = 1, renormalize: bool = True, scale: float = 1.0):
        if score not in ROUTER_SCORES:
            raise KernelError(f"unknown router score {score!r}; known: {', '.join(ROUTER_SCORES)}")
        if int(group_best) < 1:
            raise KernelError(f"a group's score is made of at least one of its outputs, not {group_best}")
        self.score, self.group_best, self.renormalize, self.scale = score, int(group_best), bool(renormalize), float(scale)

    def args(self) -> tuple:
        return ROUTER_SCORES[self.score], self.group_best, 1 if self.renormalize else 0, self.scale


_DEFAULT_RULE = RouterRule()


def _expert_act(activation: str, limit: Optional[float], gated: bool = True) -> tuple:
    known = EXPERT_ACTIVATIONS if gated else PLAIN_ACTIVATIONS
    try:
        code = known[activation]
    except KeyError:
        raise KernelError(f"unknown expert activation {activation!r}; known: {', '.join(known)}") from None
    if code == 2 and not (limit is not None and limit > 0.0):
        raise KernelError(f"the clamped activation needs a positive limit, found {limit!r}")
    return code, float(limit or 0.0)


def route_topk(logits: torch.Tensor, correction: Optional[torch.Tensor], top: int, group_count: int = 1,
               group_keep: int = 1, rule: Optional[RouterRule] = None) -> tuple:
    """The router's choice for every row of float32 ``logits [rows, outputs]``: scores softmax(logits) (or what
    ``rule`` says); choice scores with ``correction`` added; the outputs form ``group_count`` equal groups of
    neighbours of which the ``group_keep`` with the best group score stay open; the ``top`` best open outputs win.
    Returns their indices (int32 ``[rows, top]``, best first) and their weights (float32): by default their scores
    over the winners' sum."""
    rows, total = logits.shape
    if total > library().leone_route_max_outputs():
        raise KernelError(f"route_topk: {total} router outputs, the kernel takes {library().leone_route_max_outputs()}")
    chosen = torch.empty((rows, top), dtype=torch.int32, device=logits.device)
    weight = torch.empty((rows, top), dtype=torch.float32, device=logits.device)
    call("leone_route_topk", _dev(logits, "router logits", torch.float32),
         _dev(correction, "router correction", None, (total,)), _code(correction, "router correction") if correction is not None else F32,
         _dev(chosen, "chosen"), _dev(weight, "weights"), rows, total, int(top), int(group_count), int(group_keep),
         *(rule or _DEFAULT_RULE).args(), _stream())
    return chosen, weight


MOE_WIDE_TILE_PAIRS = 32      # from this many (row, place) pairs an expert on average, the experts' products take tiles of 64 pairs
ROUTE_PLAN_ROWS = 64          # up to here the router's choice and the tiles are made in one launch


def _expert_tiles(x: torch.Tensor, rows: int, top: int, experts: int, hidden: int, ff: int):
    """(pairs a tile, tiles at most, tile_expert, tile_pairs) for a step of ``rows`` rows."""
    pairs = rows * top
    # bfloat16 with inner sizes in runs of 8 goes to the matrix cores: tiles of 128 or 64 pairs where an expert gets
    # many (its matrices are read once a tile), of 16 where it gets few; anything else in tiles of the plain kernel's size
    if x.dtype == torch.bfloat16 and hidden % 8 == 0 and ff % 8 == 0:
        tile = 128 if pairs >= 4 * MOE_WIDE_TILE_PAIRS * experts else 64 if pairs >= MOE_WIDE_TILE_PAIRS * experts else 16
    else:
        tile = library().leone_moe_tile_pairs()
    max_tiles = min(pairs, pairs // tile + experts)
    return (tile, max_tiles, torch.empty((max_tiles,), dtype=torch.int32, device=x.device),
            torch.empty((max_tiles, tile), dtype=torch.int32, device=x.device))


def _check_experts(x: torch.Tensor, w_up: torch.Tensor, w_down: torch.Tensor):
    """(rows, hidden, experts, ff, whether the experts have a gate)."""
    rows, hidden = x.shape
    gated = w_up.dim() == 4
    experts, ff, k = w_up.shape[0], w_up.shape[-2], w_up.shape[-1]
    if w_up.dim() not in (3, 4) or (gated and w_up.shape[1] != 2) or k != hidden or tuple(w_down.shape) != (experts, hidden, ff) \
            or w_up.dtype != x.dtype or w_down.dtype != x.dtype:
        raise KernelError(f"routed experts: matrices {tuple(w_up.shape)} and {tuple(w_down.shape)} of {w_up.dtype} "
                          f"do not fit rows {tuple(x.shape)} of {x.dtype}")
    return rows, hidden, experts, ff, gated


def _expert_products(x, chosen, weight, tiles, w_up, w_down, activation, extra, limit=None, weigh_input=False) -> torch.Tensor:
    rows, hidden, experts, ff, gated = _check_experts(x, w_up, w_down)
    if weigh_input and gated:
        raise KernelError("routed experts: a weight on what an expert reads goes with experts without a gate")
    act, limit = _expert_act(activation, limit, gated)
    top = chosen.shape[1]
    pairs = rows * top
    tile, max_tiles, tile_expert, tile_pairs = tiles
    device = x.device
    weights = _dev(weight, "weights", torch.float32, (rows, top))
    hidden_act = torch.empty((pairs, ff), dtype=x.dtype, device=device)
    # the weight stands on the input's side (a product of weight * x is weight times the product) or on the result's
    call("leone_moe_product", _dev(x, "routed rows"), _dev(w_up, "expert up"), _dev(hidden_act, "expert hidden"),
         weights if weigh_input else 0, _code(x, "routed rows"), 1 if gated else 2, _dev(tile_expert, "tiles"),
         _dev(tile_pairs, "tile pairs"), max_tiles, tile, top, ff, hidden, act, limit, _stream())
    pair_out = torch.empty((pairs, hidden), dtype=torch.float32, device=device)
    call("leone_moe_product", _dev(hidden_act, "expert hidden"), _dev(w_down, "expert down"), _dev(pair_out, "pair results"),
         0 if weigh_input else weights, _code(x, "routed rows"), 0, _dev(tile_expert, "tiles"),
         _dev(tile_pairs, "tile pairs"), max_tiles, tile, top, hidden, ff, 0, 0.0, _stream())
    out = torch.empty((rows, hidden), dtype=torch.float32, device=device)
    call("leone_moe_combine", _dev(pair_out, "pair results"), _dev(chosen, "chosen"), weights,
         _dev(x, "routed rows"), _code(x, "routed rows"), _dev(extra, "extra", torch.float32, (rows, hidden)),
         _dev(out, "routed out"), rows, top, experts, hidden, _stream())
    return out


def routed_experts(x: torch.Tensor, chosen: torch.Tensor, weight: torch.Tensor, w_gate_up: torch.Tensor,
                   w_down: torch.Tensor, activation: str = "silu", extra: Optional[torch.Tensor] = None,
                   limit: Optional[float] = None, weigh_input: bool = False) -> torch.Tensor:
    """Every row through the experts chosen for it: float32 ``[rows, hidden]`` = sum over a row's places of
    weight * W_down[e] (act(W_gate[e] x) * (W_up[e] x)), in the places' order; a chosen index from the number of
    experts on stands for an expert that hands the row on as it is; ``extra`` (float32 ``[rows, hidden]``) is added.
    ``w_gate_up`` is ``[experts, 2, ff, hidden]`` (gate rows, then up rows), ``w_down`` ``[experts, hidden, ff]``, both
    of ``x``'s type; experts without a gate come as ``[experts, ff, hidden]`` and compute W_down[e] act(W_up[e] x)
    (``PLAIN_ACTIVATIONS``).  ``weigh_input`` (experts without a gate): the weight multiplies what the expert reads
    instead of what it gives.  Nothing here depends on the choice except through device arrays."""
    rows, hidden, experts, ff, _ = _check_experts(x, w_gate_up, w_down)
    top = chosen.shape[1]
    tiles = _expert_tiles(x, rows, top, experts, hidden, ff)
    call("leone_moe_plan", _dev(chosen, "chosen", torch.int32, (rows, top)), rows * top, experts, _dev(tiles[2], "tiles"),
         _dev(tiles[3], "tile pairs"), tiles[1], tiles[0], _stream())
    return _expert_products(x, chosen, weight, tiles, w_gate_up, w_down, activation, extra, limit, weigh_input)


def routed_feed_forward(x: torch.Tensor, logits: torch.Tensor, correction: Optional[torch.Tensor], top: int, group_count: int,
                        group_keep: int, w_gate_up: torch.Tensor, w_down: torch.Tensor, activation: str = "silu",
                        extra: Optional[torch.Tensor] = None, always: int = 0, rule: Optional[RouterRule] = None,
                        limit: Optional[float] = None, weigh_input: bool = False) -> torch.Tensor:
    """``route_topk`` on the router's float32 ``logits`` and ``routed_experts`` with its choice; for steps of few rows
    (up to ``ROUTE_PLAN_ROWS``) the choice and the tiles are made in one launch.  ``always`` (such steps only): the
    last so many experts of the matrices are no choice of the router's but taken by every row with weight 1 (a
    shared expert cut to the experts' size rides along in the experts' launches)."""
    rows, hidden, experts, ff, _ = _check_experts(x, w_gate_up, w_down)
    total = logits.shape[1]
    if rows > ROUTE_PLAN_ROWS:
        if always:
            raise KernelError(f"routed_feed_forward: experts for every row ride along in steps of up to {ROUTE_PLAN_ROWS} rows only")
        chosen, weight = route_topk(logits, correction, top, group_count, group_keep, rule)
        return routed_experts(x, chosen, weight, w_gate_up, w_down, activation, extra, limit, weigh_input)
    if total > library().leone_route_max_outputs():
        raise KernelError(f"route_topk: {total} router outputs, the kernel takes {library().leone_route_max_outputs()}")
    if not 0 <= always < experts:
        raise KernelError(f"routed_feed_forward: {always} of {experts} experts for every row")
    places = top + always
    tiles = _expert_tiles(x, rows, places, experts, hidden, ff)
    chosen = torch.empty((rows, places), dtype=torch.int32, device=x.device)
    weight = torch.empty((rows, places), dtype=torch.float32, device=x.device)
    call("leone_route_plan", _dev(logits, "router logits", torch.float32, (rows, total)),
         _dev(correction, "router correction", None, (total,)), _code(correction, "router correction") if correction is not None else F32,
         _dev(chosen, "chosen"), _dev(weight, "weights"), rows, total, int(top), int(group_count), int(group_keep), experts,
         _dev(tiles[2], "tiles"), _dev(tiles[3], "tile pairs"), tiles[1], tiles[0], int(always),
         *(rule or _DEFAULT_RULE).args(), _stream())
    return _expert_products(x, chosen, weight, tiles, w_gate_up, w_down, activation, extra, limit, weigh_input)


# ---- a forget gate per key channel, attention through a shared latent, the stream as a sum over depth -----------
GATED_CHUNKS = (64, 256)     # rows of a chunk and the portions that are walked in chunks (as ``OUTER_CHUNKS``)


def gated_scan(proj: torch.Tensor, columns: dict, f_bias: torch.Tensor, lower: torch.Tensor, state: torch.Tensor, step,
               heads: int, dim: int, vdim: int, q_activation: Optional[str] = "silu", write_state: bool = True) -> torch.Tensor:
    """The matrix memory whose forget gate also says what is written, over every entry's rows: per head and key
    channel f = lower + (1 - lower) sigmoid(pre + f_bias); S <- diag(f) S + (1 - f) v^T; o = S^T q with q = act(q_pre).
    ``proj`` float32 ``[rows, width]`` holds q_pre, the gates' pre (``heads * dim`` each) and v (``heads * vdim``) at
    ``columns`` "q", "f", "v"; ``f_bias`` and ``lower`` ``[heads * dim]`` of one type; ``state`` float32
    ``[slots, heads, dim * vdim]``.  Returns o float32 ``[rows, heads * vdim]``.  Long portions are walked in chunks
    side by side, as in ``outer_scan``, the chunks chained by the product of their gates per key channel."""
    rows, width = proj.shape
    if state.dtype != torch.float32 or state.dim() != 3 or tuple(state.shape[1:]) != (heads, dim * vdim) or not state.is_contiguous():
        raise KernelError(f"gated_scan: state {tuple(state.shape)} is not [slots, {heads}, {dim * vdim}] float32")
    if f_bias.dtype != lower.dtype:
        raise KernelError("gated_scan: the gates' bias and lower bound must share one type")
    if q_activation not in (None, "silu"):
        raise KernelError(f"gated_scan: queries pass as they are or through silu, not {q_activation!r}")
    out = torch.empty((rows, heads * vdim), dtype=torch.float32, device=proj.device)

    def walk(segments, state_in, state_out, no_input=False, accumulate=False, product=None):
        call("leone_gated_scan", _dev(proj, "projection", torch.float32), width, columns["q"], columns["f"], columns["v"],
             _dev(f_bias, "gate bias", None, (heads * dim,)), _dev(lower, "lower bound", None, (heads * dim,)),
             _code(f_bias, "gate bias"), 1 if q_activation == "silu" else 0, 1 if no_input else 0, 1 if accumulate else 0,
             _dev(segments, "segments", torch.int32), segments.shape[0],
             _dev(state_in, "state read"), state_in.stride(0) if state_in is not None else 0,
             _dev(state_out, "state written"), state_out.stride(0) if state_out is not None else 0,
             _dev(product, "gate products"), _dev(out, "out"), heads, dim, vdim, _stream())

    _walk_rows(step, walk, state, heads, dim, vdim, write_state)
    return out


def state_space_scan(xbc: torch.Tensor, columns: dict, groups: int, step_size: torch.Tensor, step_bias: torch.Tensor,
                     rate_log: torch.Tensor, skip: torch.Tensor, state: torch.Tensor, step, heads: int, dim: int, vdim: int,
                     write_state: bool = True) -> torch.Tensor:
    """A state-space layer's recurrence over every entry's rows: per head, with dt = softplus(pre + step_bias),
    S <- exp(-exp(rate_log) dt) S + (dt B) x^T (S is ``dim`` x ``vdim``), o = S^T C + skip x.  ``xbc`` float32
    ``[rows, width]`` holds x (``heads * vdim`` columns from ``columns["x"]``), B and C (``groups * dim`` columns each from
    "b" and "c"; head h reads group h // (heads / groups)); ``step_size`` float32 ``[rows, >= heads]`` the step sizes'
    pre-activations (a slice of wider rows is fine); ``step_bias``, ``rate_log``, ``skip`` ``[heads]`` of one type;
    ``state`` float32 ``[slots, heads, dim * vdim]``.  Returns o float32 ``[rows, heads * vdim]``.  Long portions are walked
    in chunks side by side, as in ``gated_scan``, chained by the product of the chunk's decays."""
    rows, width = xbc.shape
    if state.dtype != torch.float32 or state.dim() != 3 or tuple(state.shape[1:]) != (heads, dim * vdim) or not state.is_contiguous():
        raise KernelError(f"state_space_scan: state {tuple(state.shape)} is not [slots, {heads}, {dim * vdim}] float32")
    if len({step_bias.dtype, rate_log.dtype, skip.dtype}) != 1:
        raise KernelError("state_space_scan: the step bias, the rates' logarithms and the skip weights must share one type")
    if groups <= 0 or heads % groups:
        raise KernelError(f"state_space_scan: {heads} heads do not share {groups} groups evenly")
    step_at, step_stride = _strided_rows(step_size, "step sizes", rows, heads)
    out = torch.empty((rows, heads * vdim), dtype=torch.float32, device=xbc.device)

    def walk(segments, state_in, state_out, no_input=False, accumulate=False, product=None):
        call("leone_state_space_scan", _dev(xbc, "x, B and C", torch.float32), width, columns["x"], columns["b"], columns["c"],
             groups, step_at, step_stride, 0, _dev(step_bias, "step bias", None, (heads,)),
             _dev(rate_log, "rate logarithms", None, (heads,)), _dev(skip, "skip weights", None, (heads,)),
             _code(step_bias, "step bias"), 1 if no_input else 0, 1 if accumulate else 0,
             _dev(segments, "segments", torch.int32), segments.shape[0],
             _dev(state_in, "state read"), state_in.stride(0) if state_in is not None else 0,
             _dev(state_out, "state written"), state_out.stride(0) if state_out is not None else 0,
             _dev(product, "decay products"), _dev(out, "out"), heads, dim, vdim, _stream())

    _walk_rows(step, walk, state, heads, dim, vdim, write_state)
    return out


def time_mix_scan(r: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: torch.Tensor, bonus: torch.Tensor,
                  state: torch.Tensor, step, heads: int, dim: int, vdim: int, write_state: bool = True) -> torch.Tensor:
    """A matrix memory with ready-made decays over every entry's rows: per head o_t = (S + diag(bonus) k_t v_t^T)^T r_t,
    then S <- diag(decay_t) S + k_t v_t^T.  ``r``, ``k`` (``heads * dim`` columns) and ``v`` (``heads * vdim``) are float32
    rows, possibly slices of wider rows, all with one distance from row to row; ``decay`` float32 ``[rows, heads * dim]``;
    ``bonus`` ``[heads * dim]``; ``state`` float32 ``[slots, heads, dim * vdim]``.  Returns o float32 ``[rows, heads * vdim]``.
    Long portions are walked in chunks side by side, as in ``gated_scan``, chained by the product of the chunk's decays."""
    rows = r.shape[0]
    if state.dtype != torch.float32 or state.dim() != 3 or tuple(state.shape[1:]) != (heads, dim * vdim) or not state.is_contiguous():
        raise KernelError(f"time_mix_scan: state {tuple(state.shape)} is not [slots, {heads}, {dim * vdim}] float32")
    r_at, stride = _strided_rows(r, "r", rows, heads * dim)
    k_at, k_stride = _strided_rows(k, "k", rows, heads * dim)
    v_at, v_stride = _strided_rows(v, "v", rows, heads * vdim)
    if not stride == k_stride == v_stride:
        raise KernelError(f"time_mix_scan: r, k and v lie {stride}, {k_stride} and {v_stride} elements apart from row to row")
    out = torch.empty((rows, heads * vdim), dtype=torch.float32, device=r.device)

    single_rows = bool(step.decode_only) and step.entry_slots.numel() == rows

    def walk(segments, state_in, state_out, product=None):
        call("leone_time_mix_scan", r_at, k_at, v_at, stride, _dev(decay, "decays", torch.float32, (rows, heads * dim)),
             _dev(bonus, "bonus", None, (heads * dim,)), _code(bonus, "bonus"), _dev(segments, "segments", torch.int32),
             segments.shape[0], 1 if single_rows else 0,
             _dev(state_in, "state read"), state_in.stride(0) if state_in is not None else 0,
             _dev(state_out, "state written"), state_out.stride(0) if state_out is not None else 0,
             _dev(product, "decay products"), _dev(out, "out"), heads, dim, vdim, _stream())

    def read(segments, work):
        call("leone_time_mix_read", r_at, stride, _dev(decay, "decays", torch.float32, (rows, heads * dim)),
             _dev(segments, "segments", torch.int32), segments.shape[0], _dev(work, "chunk states"), work.stride(0),
             _dev(out, "out"), heads, dim, vdim, _stream())

    chunk = min(GATED_CHUNKS[0], library().leone_time_mix_read_rows())
    _walk_rows(step, walk, state, heads, dim, vdim, write_state, read=read, chunks=(chunk, GATED_CHUNKS[1]))
    return out


def token_mix(h: torch.Tensor, mu: torch.Tensor, state: torch.Tensor, step, write_state: bool = True) -> torch.Tensor:
    """h + (h' - h) * mu[m] for every vector of ``mu`` ``[mixes, hidden]``, h' the token before of the same request: the row
    above, the request's stored row (``state`` float32 ``[slots, hidden]``) ahead of a portion, zeros at a sequence's
    start.  Returns ``[mixes, rows, hidden]`` in ``h``'s type and stores every entry's last row unless told not to."""
    rows, hidden = h.shape
    mixes = mu.shape[0]
    if tuple(mu.shape) != (mixes, hidden) or state.dtype != torch.float32 or tuple(state.shape[1:]) != (hidden,):
        raise KernelError(f"token_mix: mixes {tuple(mu.shape)} and state {tuple(state.shape)} for rows of {hidden}")
    spans = entry_spans(step)
    out = torch.empty((mixes, rows, hidden), dtype=h.dtype, device=h.device)
    single_rows = bool(step.decode_only) and step.entry_slots.numel() == rows
    call("leone_token_mix", _dev(h, "rows"), _code(h, "rows"), _dev(mu, "mu"), _code(mu, "mu"), mixes, _dev(state, "stored rows"),
         state.data_ptr() if write_state else 0, _dev(spans, "spans"), spans.shape[0],
         _dev(step.row_entry, "row map", torch.int32, (rows,)), _dev(out, "mixed rows"), rows, hidden, 1 if single_rows else 0, _stream())
    return out


def low_rank_decay(low: torch.Tensor, w2: torch.Tensor, w0: torch.Tensor) -> torch.Tensor:
    """exp(-exp(w2 tanh(low) + w0)): ``low`` float32 ``[rows, >= rank]`` (a slice of wider rows is fine), ``w2``
    ``[channels, rank]``, ``w0`` ``[channels]`` -> float32 ``[rows, channels]``, all of it float."""
    channels, rank = w2.shape
    rows = low.shape[0]
    low_at, stride = _strided_rows(low, "low-rank values", rows, rank)
    out = torch.empty((rows, channels), dtype=torch.float32, device=low.device)
    call("leone_low_rank_decay", low_at, stride, _dev(w2, "decay matrix"), _code(w2, "decay matrix"),
         _dev(w0, "decay base", None, (channels,)), _code(w0, "decay base"), _dev(out, "decays"), rows, channels, rank, _stream())
    return out


def _walk_rows(step, walk, state: torch.Tensor, heads: int, dim: int, vdim: int, write_state: bool, read=None,
               chunks: Optional[tuple] = None) -> None:
    """A recurrence S <- diag(decay) S + ... over a step's rows: ``walk(segments, state read, state written, no_input=,
    accumulate=, product=)`` walks segments of rows in order.  Long portions go chunk by chunk side by side: every chunk
    from zeros (leaving what it wrote and the product of its decays), the chunks chained, every chunk again from the
    state it starts from with nothing written into it (by ``read(segments, states)`` if the recurrence has such a kernel).
    ``chunks``: rows of a chunk and the portions walked so, ``GATED_CHUNKS`` if not said."""
    plan = chunk_plan(step, *(chunks or GATED_CHUNKS))
    if plan is None:
        walk(entry_spans(step), state, state if write_state else None)
        return
    listed = plan["chunks"]
    work = torch.empty((listed.shape[0], heads, dim * vdim), dtype=torch.float32, device=state.device)
    product = torch.empty((listed.shape[0], heads, dim), dtype=torch.float32, device=state.device)
    walk(listed, None, work, product=product)
    call("leone_gated_chain", _dev(plan["links"], "links", torch.int32), plan["links"].shape[0], _dev(work, "work"),
         work.stride(0), _dev(product, "decay products"), _dev(state, "state"), state.stride(0), heads, dim, vdim,
         1 if write_state else 0, _stream())
    if read is not None:
        read(plan["again"], work)
    else:
        walk(plan["again"], work, None, no_input=True, accumulate=True)
    if plan["short"].shape[0]:
        walk(plan["short"], state, state if write_state else None)


def _rotation_tables(what: str, part: int, cos, sin):
    """(address of cos, of sin, pairs, table positions) of a rotation of neighbouring pairs on the first elements of a
    part of ``part`` elements."""
    if cos is None:
        return 0, 0, 0, 1
    if sin is None or sin.shape != cos.shape or cos.dim() != 2 or 2 * cos.shape[1] > part:
        raise KernelError(f"{what}: cos and sin tables must both be [positions, pairs] with 2 * pairs <= {part}")
    return _dev(cos, "rope cos", torch.float32), _dev(sin, "rope sin", torch.float32), cos.shape[1], cos.shape[0]


def latent_prepare(proj: torch.Tensor, out_dtype: torch.dtype, eps: float, *, q_column: Optional[int] = None, q_rank: int = 0,
                   q_gain: Optional[torch.Tensor] = None, kv_column: Optional[int] = None, rank: int = 0, rot: int = 0,
                   kv_gain: Optional[torch.Tensor] = None, cos: Optional[torch.Tensor] = None,
                   sin: Optional[torch.Tensor] = None, positions: Optional[torch.Tensor] = None,
                   row_entry: Optional[torch.Tensor] = None, block_table: Optional[torch.Tensor] = None,
                   k_pool: Optional[torch.Tensor] = None, v_pool: Optional[torch.Tensor] = None) -> Optional[torch.Tensor]:
    """From the float32 down-projections ``proj [rows, width]``: the query latent (``q_rank`` columns from
    ``q_column``) RMS-normed times ``q_gain`` comes back in ``out_dtype``; the key/value latent (``rank`` columns from
    ``kv_column``) RMS-normed times ``kv_gain`` and the ``rot`` columns behind it, rotated in neighbouring pairs by the
    row's position, are written at the row's place into the cache: as a key into ``k_pool [pages, ceil((rank + rot) / 8),
    page_tokens, 8]`` and the latent once more as a value into ``v_pool [pages, page_tokens / 8, rank, 8]``.  Either half
    may be left out."""
    rows, width = proj.shape
    q_out = torch.empty((rows, q_rank), dtype=out_dtype, device=proj.device) if q_column is not None else None
    gains = [g for g in (q_gain, kv_gain) if g is not None]
    if not gains or len({g.dtype for g in gains}) != 1:
        raise KernelError("latent_prepare: the gains must come in one type")
    page_tokens = max_blocks = 0
    if kv_column is not None:
        page_tokens = _latent_pools("latent_prepare", k_pool, v_pool, rank, rot, out_dtype)
        if block_table is None or positions is None or row_entry is None:
            raise KernelError("latent_prepare: a cache write needs positions, a row map and a block table")
        max_blocks = block_table.shape[1]
    cos_at, sin_at, pairs, table_positions = _rotation_tables("latent_prepare", rot, cos, sin)
    call("leone_latent_prepare", _dev(proj, "projection", torch.float32), width, rows,
         -1 if q_column is None else int(q_column), int(q_rank), _dev(q_gain, "query gain", None, (q_rank,)) if q_column is not None else 0,
         _dev(q_out, "query latent"), -1 if kv_column is None else int(kv_column), int(rank), int(rot),
         _dev(kv_gain, "latent gain", None, (rank,)) if kv_column is not None else 0, _code(gains[0], "gain"), float(eps),
         cos_at, sin_at, pairs, table_positions,
         _dev(positions, "positions", torch.int32, (rows,)) if kv_column is not None else 0,
         _dev(row_entry, "row map", torch.int32, (rows,)) if kv_column is not None else 0,
         _dev(block_table, "block table", torch.int32) if kv_column is not None else 0, max_blocks, page_tokens,
         _dev(k_pool, "latent keys") if kv_column is not None else 0, _dev(v_pool, "latent values") if kv_column is not None else 0,
         _CODES[out_dtype], _stream())
    return q_out


def _latent_pools(what: str, k_pool, v_pool, rank: int, rot: int, dtype) -> int:
    """Checks the two forms of a latent cache against each other and the sizes; returns the tokens a page holds."""
    runs = -(-(rank + rot) // 8)
    if k_pool is None or v_pool is None or k_pool.dim() != 4 or v_pool.dim() != 4 or k_pool.shape[1] != runs or k_pool.shape[3] != 8 \
            or tuple(v_pool.shape) != (k_pool.shape[0], k_pool.shape[2] // 8, rank, 8) or k_pool.shape[2] % 8 \
            or k_pool.dtype != v_pool.dtype or (dtype is not None and k_pool.dtype != dtype):
        raise KernelError(f"{what}: the cache must be [pages, {runs}, page_tokens, 8] and [pages, page_tokens / 8, {rank}, 8] of one "
                          f"type, found {None if k_pool is None else (k_pool.dtype, tuple(k_pool.shape))} and "
                          f"{None if v_pool is None else (v_pool.dtype, tuple(v_pool.shape))}")
    return k_pool.shape[2]


HEAD_PRODUCT_LIBRARY_ROWS = 128      # from here on a bfloat16 product a head goes to the library's batched product


def head_product(x: torch.Tensor, weight: torch.Tensor, heads: int, out_dtype: torch.dtype, *, tail: int = 0,
                 cos: Optional[torch.Tensor] = None, sin: Optional[torch.Tensor] = None,
                 positions: Optional[torch.Tensor] = None) -> torch.Tensor:
    """A product a head: ``x`` float32 ``[rows, heads * (inner + tail)]``, ``weight`` ``[heads, inner, outer]`` ->
    ``[rows, heads * (outer + tail)]`` in ``out_dtype`` with y[r, h, :outer] = x[r, h, :inner] weight[h] (``x`` may be a
    column slice of wider rows).  The ``tail``
    elements behind a head's inner ones are handed on behind its outer ones, rotated in neighbouring pairs by the
    row's position if tables come.  Many rows of a bfloat16 model go through the library's batched product (the rows
    rounded to bfloat16, float accumulation); the kernel then hands on the tails alone."""
    rows = x.shape[0]
    if weight.dim() != 3 or weight.shape[0] != heads or x.dim() != 2 or x.shape[1] != heads * (weight.shape[1] + tail):
        raise KernelError(f"head_product: rows {tuple(x.shape)} against {tuple(weight.shape)} for {heads} heads with a tail of {tail}")
    inner, outer = weight.shape[1], weight.shape[2]
    out = torch.empty((rows, heads * (outer + tail)), dtype=out_dtype, device=x.device)
    cos_at, sin_at, pairs, table_positions = _rotation_tables("head_product", tail, cos, sin)
    library = weight.dtype == torch.bfloat16 and rows >= HEAD_PRODUCT_LIBRARY_ROWS and inner % 8 == 0 and outer % 8 == 0
    if library:
        with profile.span(profile.LIBRARY_PRODUCT, weight):
            part = x.view(rows, heads, inner + tail)[:, :, :inner]
            if part.dtype != torch.bfloat16:
                part = part.to(torch.bfloat16)
            y = torch.bmm(part.transpose(0, 1), weight) if out_dtype == torch.bfloat16 else \
                torch.bmm(part.transpose(0, 1), weight, out_dtype=torch.float32)
            out.view(rows, heads, outer + tail)[:, :, :outer].copy_(y.transpose(0, 1))
        if not tail:
            return out
    x_at, x_stride = _strided_rows(x, "head rows", rows, x.shape[1])
    call("leone_head_product", x_at, x_stride, inner + tail,
         0 if library else _dev(weight, "head matrices"), _code(weight, "head matrices"), _dev(out, "head results"),
         _CODES[out_dtype], out.shape[1], outer + tail, rows, heads,
         inner, outer, int(tail), cos_at, sin_at, pairs, table_positions,
         _dev(positions, "positions", torch.int32, (rows,)) if cos is not None else 0, _stream())
    return out


def latent_cores_supported(dtype: torch.dtype, rank: int, rot: int, page_tokens: int) -> bool:
    """Whether the matrix-core kernel takes a latent cache of these sizes; otherwise the kernel for any size does."""
    return (dtype == torch.bfloat16 and (rank + rot) % 32 == 0 and rank % 16 == 0 and page_tokens % 32 == 0
            and rank + rot <= library().leone_latent_cores_max_width())


LATENT_SPLIT_TILES = 1       # a wave of the matrix-core kernel keeps at least this many 32-key tiles when keys are shared out
LATENT_MAX_SPLITS = 16


def latent_splits(pairs: int, keys: int, units: int = 256) -> int:
    """How many workgroups share the keys of every 16 (row, head) pairs: one where the tiles of pairs fill the GPU by
    themselves, more in steps of few rows over long contexts."""
    tiles = -(-pairs // 16)
    by_room = units // max(tiles, 1)
    by_work = -(-(-(-keys // 32) + 1) // (4 * LATENT_SPLIT_TILES))       # a range of keys seldom begins with a tile: one more
    return max(1, min(by_room, by_work, LATENT_MAX_SPLITS))


def latent_attention(q: torch.Tensor, k_pool: torch.Tensor, v_pool: torch.Tensor, positions: torch.Tensor,
                     row_entry: torch.Tensor, block_table: torch.Tensor, heads: int, rank: int, rot: int, scale: float,
                     window: int = 0, max_position: Optional[int] = None) -> torch.Tensor:
    """Softmax attention over a cache of latents shared by the heads: ``q`` ``[rows, heads * (rank + rot)]`` (the keys'
    up-projection already on the query's side, see ``head_product``), the cache in its two forms (``latent_prepare``);
    a row sees the latents of its request at positions pos - window < j <= pos (``window`` 0: all).  Returns float32
    ``[rows, heads * rank]``: every head's weighted sum of the latents.  bfloat16 queries go to the matrix-core kernel
    (``latent_cores_supported``), float32 queries to the kernel for any size and type of cache.  ``max_position``: the
    largest position in the step or a bound on it, known on the host: few rows over many keys are shared out over
    several workgroups by it (``latent_splits``)."""
    rows = q.shape[0]
    page_tokens = _latent_pools("latent_attention", k_pool, v_pool, rank, rot, None)
    if q.shape[1] != heads * (rank + rot):
        raise KernelError(f"latent_attention: queries {tuple(q.shape)} do not fit {heads} heads of {rank} + {rot}")
    out = torch.empty((rows, heads * rank), dtype=torch.float32, device=q.device)
    if q.dtype == torch.bfloat16:
        if not latent_cores_supported(k_pool.dtype, rank, rot, page_tokens):
            raise KernelError(f"latent_attention: bfloat16 queries are for the matrix-core kernel, which does not take a "
                              f"{k_pool.dtype} cache of {rank} + {rot} in pages of {page_tokens}")
        keys = 0 if max_position is None else (min(int(window), max_position + 1) if window else max_position + 1)
        splits = latent_splits(rows * heads, keys, compute_units(q.device))
        part_acc = part_ml = None
        if splits > 1:
            tiles = -(-rows * heads // 16)
            part_acc = torch.empty((tiles, splits, 16, rank), dtype=torch.float32, device=q.device)
            part_ml = torch.empty((tiles, splits, 16, 2), dtype=torch.float32, device=q.device)
        call("leone_latent_attention_cores", _dev(q, "latent queries", torch.bfloat16), _dev(out, "latent sums"),
             _dev(k_pool, "latent keys"), _dev(v_pool, "latent values"), _dev(positions, "positions", torch.int32, (rows,)),
             _dev(row_entry, "row map", torch.int32, (rows,)), _dev(block_table, "block table", torch.int32),
             block_table.shape[1], rows, heads, int(rank), int(rot), page_tokens, float(scale), int(window), splits,
             _dev(part_acc, "partial sums"), _dev(part_ml, "partial maxima"), _stream())
        return out
    if rank + rot > library().leone_latent_max_width():
        raise KernelError(f"latent_attention: a latent of {rank} + {rot} elements, the kernel takes {library().leone_latent_max_width()}")
    call("leone_latent_attention", _dev(q, "latent queries", torch.float32), _dev(out, "latent sums"), _dev(k_pool, "latent keys"),
         _code(k_pool, "latent keys"), _dev(positions, "positions", torch.int32, (rows,)),
         _dev(row_entry, "row map", torch.int32, (rows,)), _dev(block_table, "block table", torch.int32), block_table.shape[1],
         rows, heads, int(rank), int(rot), page_tokens, float(scale), int(window), _stream())
    return out


class ScaledDelta:
    """What a sublayer adds to the stream, still to be multiplied by a factor: ``scale * rows`` is meant (``rows``
    float32 ``[n, hidden]`` or planes ``[p, n, hidden]``).  The norm that runs next takes it in place of a delta
    (``residual_norm``); any other consumer asks for ``materialize()``."""

    def __init__(self, rows: torch.Tensor, scale: float):
        self.rows, self.scale = rows, float(scale)

    def materialize(self) -> torch.Tensor:
        rows = self.rows.sum(dim=0) if self.rows.dim() == 3 else self.rows
        return rows.float() * self.scale


def _planes(delta: Optional[torch.Tensor], n: int, hidden: int, what: str):
    if delta is None:
        return None, 1, 0
    if delta.dtype != torch.float32:
        delta = delta.float()
    stacked = delta.dim() == 3
    planes = delta.shape[0] if stacked else 1
    _dev(delta, what, torch.float32, (planes, n, hidden) if stacked else (n, hidden))
    return delta, planes, n * hidden


def residual_norm(x: torch.Tensor, delta: Optional[torch.Tensor], scale: float, gain: Optional[torch.Tensor], eps: float,
                  out_dtype: Optional[torch.dtype], rows: Optional[torch.Tensor] = None) -> Optional[torch.Tensor]:
    """x += scale * delta in the float32 stream (``delta`` float32 ``[n, hidden]`` or planes; None: nothing is added), then
    rmsnorm(x) * gain in ``out_dtype`` (None: no norm, only the sum).  With ``rows`` (int32 indices) only those rows come
    back and the stream is left as it was."""
    n, hidden = x.shape
    delta, planes, plane = _planes(delta, n, hidden, "delta")
    n_out = n if rows is None else rows.numel()
    y = torch.empty((n_out, hidden), dtype=out_dtype, device=x.device) if out_dtype is not None else None
    if delta is None and y is None:
        return None
    call("leone_residual_norm", _dev(x, "stream", torch.float32), _dev(delta, "delta"), planes, plane, float(scale),
         _dev(gain, "gain", None, (hidden,)) if y is not None else 0, _code(gain, "gain") if y is not None else F32, float(eps),
         _dev(y, "normed rows"), _CODES[out_dtype] if out_dtype is not None else F32,
         _dev(rows, "rows", torch.int32) if rows is not None else 0, n_out, hidden, _stream())
    return y


def depth_mix(x: torch.Tensor, delta: Optional[torch.Tensor], scale: float, history: torch.Tensor, count: int,
              weight: torch.Tensor) -> None:
    """A layer's own result X = x + scale * delta is kept as ``history[count - 1]`` and the stream becomes
    sum_{j < count} weight[j] * history[j], in place in ``x``.  ``history`` float32 ``[slots, n, hidden]``."""
    n, hidden = x.shape
    delta, planes, plane = _planes(delta, n, hidden, "delta")
    if history.dtype != torch.float32 or history.dim() != 3 or tuple(history.shape[1:]) != (n, hidden) or not 1 <= count <= history.shape[0]:
        raise KernelError(f"depth_mix: a history {tuple(history.shape)} for {count} results of {tuple(x.shape)}")
    if weight.numel() != count:
        raise KernelError(f"depth_mix: {weight.numel()} weights for {count} results")
    call("leone_depth_mix", _dev(x, "stream", torch.float32), _dev(delta, "delta"), planes, plane, float(scale),
         _dev(history, "history"), history.stride(0), int(count), _dev(weight, "depth weights"), _code(weight, "depth weights"),
         n * hidden, _stream())


# ---- sublayers side by side on one stream -----------------------------------------------------------------------
class MixedDelta:
    """What several sublayers add to the stream together: the sum of factor * scale * rows over ``terms`` = (rows float32
    ``[n, hidden]`` or planes ``[p, n, hidden]``, factor, scale vector ``[hidden]`` or None).  A norm that can takes it in
    place of a delta (``branch_norm``); any other consumer asks for ``materialize()``."""

    def __init__(self, terms):
        self.terms = list(terms)

    def materialize(self) -> torch.Tensor:
        total = None
        for rows, factor, scale in self.terms:
            rows = (rows.sum(dim=0) if rows.dim() == 3 else rows).float() * float(factor)
            rows = rows if scale is None else rows * scale.float()
            total = rows if total is None else total + rows
        return total


def delta_terms(delta) -> list:
    """What is still to be added to the stream, of any kind, as the terms of a ``MixedDelta``."""
    if delta is None or isinstance(delta, PreparedRows):
        return []
    if isinstance(delta, MixedDelta):
        return delta.terms
    if isinstance(delta, ScaledDelta):
        return [(delta.rows, delta.scale, None)]
    if isinstance(delta, NormedDelta):
        delta = delta.materialize()
    return [(delta, 1.0, None)]


def _at(array):
    return ctypes.cast(array, ctypes.c_void_p)


def _term_args(terms, n: int, hidden: int) -> tuple:
    """The arguments that name up to ``BRANCH_TERMS`` results to a kernel, and what must live until it is launched."""
    held = []
    for delta, factor, scale in terms:
        delta, planes, plane = _planes(delta, n, hidden, "result")
        held.append((delta, planes, plane, float(factor), scale))
    t = max(len(held), 1)
    term_rows = (ctypes.c_void_p * t)(*[_dev(d, "result") for d, *_ in held])
    term_planes = (ctypes.c_int * t)(*[p for _, p, *_ in held])
    term_plane = (ctypes.c_long * t)(*[p for _, _, p, *_ in held])
    factors = (ctypes.c_float * t)(*[f for *_, f, _ in held])
    scales = (ctypes.c_void_p * t)(*[_dev(s, "result scale", None, (hidden,)) for *_, s in held])
    scale_codes = (ctypes.c_int * t)(*[_code(s, "result scale") if s is not None else F32 for *_, s in held])
    return ((_at(term_rows), _at(term_planes), _at(term_plane), _at(factors), _at(scales), _at(scale_codes), len(held)),
            (held, term_rows, term_planes, term_plane, factors, scales, scale_codes))


BRANCH_TERMS = 4          # results one call adds
BRANCH_NORMS = 2          # norms it makes


def branch_norm(x: torch.Tensor, terms, gains, eps: float, groups: int, out_dtype: torch.dtype,
                rows: Optional[torch.Tensor] = None) -> list:
    """x += sum of factor * scale * rows over ``terms`` (see ``MixedDelta``) in the float32 stream, then for every gain of
    ``gains`` the RMS norm of the new rows in ``groups`` equal groups of neighbouring columns, each over its own root mean
    square, times the gain, in ``out_dtype``.  With ``rows`` (int32 indices) only those rows come back and the stream is
    left as it was."""
    n, hidden = x.shape
    terms = list(terms)
    while len(terms) > BRANCH_TERMS:                     # more than one launch takes: the first ones are added ahead
        if rows is not None:
            first = MixedDelta(terms[:len(terms) - BRANCH_TERMS + 1]).materialize()
            terms = [(first, 1.0, None)] + terms[len(terms) - BRANCH_TERMS + 1:]
        else:
            branch_norm(x, terms[:BRANCH_TERMS], [], eps, groups, out_dtype)
            terms = terms[BRANCH_TERMS:]
    if len(gains) > BRANCH_NORMS:
        raise KernelError(f"branch_norm: {len(gains)} norms, one launch makes {BRANCH_NORMS}")
    n_out = n if rows is None else rows.numel()
    outs = [torch.empty((n_out, hidden), dtype=out_dtype, device=x.device) for _ in gains]
    if not terms and not gains:
        return outs
    term_args, held = _term_args(terms, n, hidden)
    g = max(len(gains), 1)
    gain_ptrs = (ctypes.c_void_p * g)(*[_dev(v, "gain", None, (hidden,)) for v in gains])
    gain_codes = (ctypes.c_int * g)(*[_code(v, "gain") for v in gains])
    out_ptrs = (ctypes.c_void_p * g)(*[_dev(y, "normed rows") for y in outs])

    call("leone_branch_norm", _dev(x, "stream", torch.float32), *term_args, _at(gain_ptrs), _at(gain_codes), _at(out_ptrs),
         len(gains), _CODES[out_dtype], float(eps), int(groups), _dev(rows, "rows", torch.int32) if rows is not None else 0, n_out, hidden, _stream())
    return outs


def stream_join(x: torch.Tensor, terms, first: torch.Tensor, following: Optional[torch.Tensor], out_dtype: torch.dtype) -> torch.Tensor:
    """The operand ``[n, 2 hidden]`` of a product that reads the stream beside ``first`` (float32 ``[n, hidden]``): the stream's
    rows with ``terms`` (see ``MixedDelta``) added, then ``first``'s, in ``out_dtype``.  The stream ``x`` itself becomes
    ``following`` (``[hidden]``, the same for every row; None: zeros), ready for that product to be added to it."""
    n, hidden = x.shape
    terms = list(terms)
    while len(terms) > BRANCH_TERMS:
        branch_norm(x, terms[:BRANCH_TERMS], [], 1.0, 1, out_dtype)
        terms = terms[BRANCH_TERMS:]
    term_args, held = _term_args(terms, n, hidden)
    operand = torch.empty((n, 2 * hidden), dtype=out_dtype, device=x.device)
    call("leone_stream_join", _dev(x, "stream", torch.float32), *term_args, _dev(first, "first rows", torch.float32, (n, hidden)),
         _dev(following, "following rows", None, (hidden,)), _code(following, "following rows") if following is not None else F32,
         _dev(operand, "operand"), _CODES[out_dtype], n, hidden, _stream())
    return operand
