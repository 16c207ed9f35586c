"""A decoder model as data (``ModelSpec``) and the object built from it."""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional, Sequence

import torch

from .. import ops
from ..weights.loader import MATRIX, VECTOR, TensorSpec
from .base import BLOCKS, NORMS, POSITIONS, PartSpec, flatten_needs, nest_views
from .context import CacheView, StepContext


@dataclass(frozen=True)
class LayerRun:
    """One entry of the execution order.

    ``layer`` indexes ``ModelSpec.layers`` (a layer may be named more than
    once).  ``cache`` is the cache slot the run works on; two runs that name the
    same slot share it, and only runs with ``writes`` put new keys, values or
    state there.  ``borrow`` (for a layer whose cache need is a dict): name -> the
    cache slot of another run whose storage of that name this run reads without
    writing, while everything else it keeps is its own.
    """
    layer: int
    cache: Optional[int]
    writes: bool = True
    borrow: Optional[Dict[str, int]] = None

    def __hash__(self):
        return hash((self.layer, self.cache, self.writes, tuple(sorted((self.borrow or {}).items()))))


@dataclass(frozen=True)
class StreamJoin:
    """Ahead of the runs whose places in the schedule ``before`` lists, the stream becomes W [x; x0] + vectors[t]: x the stream,
    x0 the embedding's output, W the tensor ``matrix`` ``[hidden, 2 hidden]`` (x's columns first) and t the place in ``before``
    (``vectors`` ``[len(before), hidden]``).  Layers that run several times over begin every pass so."""
    before: Sequence[int]
    matrix: str
    vectors: str


@dataclass
class ModelSpec:
    hidden_size: int
    vocab_size: int
    max_positions: int
    embedding: str                                  # tensor name of the token table [vocab, hidden]
    layers: List[PartSpec]                          # block specs
    schedule: List[LayerRun]
    final_norm: PartSpec
    head: Optional[str]                             # tensor name [vocab, hidden]; None = tied to the embedding
    positions: Dict[str, PartSpec] = field(default_factory=dict)
    ignore_tensors: Sequence[str] = ()              # names a file may hold that the model does not use
    embedding_scale: Optional[float] = None         # the stream starts as table row * scale
    logit_cap: Optional[float] = None               # logits = cap * tanh(logits / cap)
    position_table: Optional[str] = None            # tensor name [max_positions, hidden]: a learned vector a position, added to the token's
    # One tensor name for every scheduled run (or None): behind run i the stream becomes the sum over j <= i + 1 of
    # weight_i[j] * X_j, with X_0 the embedding's output and X_(j+1) run j's own result; weight_i has i + 2 elements.
    depth_weights: Optional[Sequence[str]] = None
    join: Optional["StreamJoin"] = None             # where runs start from the stream and the embedding's output together


def default_schedule(n_layers: int) -> List[LayerRun]:
    return [LayerRun(i, i, True) for i in range(n_layers)]


class DecoderModel:
    """Embedding, the scheduled layer runs, final norm and the output head."""

    def __init__(self, spec: ModelSpec, dtype: torch.dtype, device):
        if dtype not in (torch.float32, torch.bfloat16):
            raise ValueError(f"engine type must be float32 or bfloat16, found {dtype}")
        self.spec = spec
        self.dtype = dtype
        self.device = torch.device(device)
        self.positions = {name: POSITIONS.build(s) for name, s in spec.positions.items()}
        self.layers = [BLOCKS.build(s, positions=self.positions) for s in spec.layers]
        self.final_norm = NORMS.build(spec.final_norm)
        self.schedule = list(spec.schedule)
        for run in self.schedule:
            if not 0 <= run.layer < len(self.layers):
                raise ValueError(f"schedule names layer {run.layer}, the model has {len(self.layers)}")
        if spec.depth_weights is not None and len(spec.depth_weights) != len(self.schedule):
            raise ValueError(f"{len(spec.depth_weights)} depth weights for {len(self.schedule)} layer runs")
        self.joins: Dict[int, int] = {}                   # run -> place among the joins
        if spec.join is not None:
            if spec.depth_weights is not None:
                raise ValueError("a stream that is joined with the embedding's output is not re-mixed over depth as well")
            self.joins = {int(run): t for t, run in enumerate(spec.join.before)}
            if len(self.joins) != len(spec.join.before) or not all(0 <= run < len(self.schedule) for run in self.joins):
                raise ValueError(f"the stream is joined ahead of runs {list(spec.join.before)}; the schedule has {len(self.schedule)}")
        self.join_matrix: Optional[torch.Tensor] = None
        self.join_vectors: List[torch.Tensor] = []
        self.depth_weights: Optional[List[torch.Tensor]] = None
        self.embedding: Optional[torch.Tensor] = None
        self.position_table: Optional[torch.Tensor] = None
        self.head: Optional[torch.Tensor] = None
        self.streamed_copy_bytes: Optional[int] = None    # None: not decided yet (``keep_streamed_copies``)

    @property
    def graph_safe(self) -> bool:
        """Whether a step of this model can be recorded once and replayed (see ``Part.graph_safe``)."""
        return (all(getattr(layer, "graph_safe", False) for layer in self.layers)
                and getattr(self.final_norm, "graph_safe", False))

    # ---- weights -------------------------------------------------------------
    def tensor_specs(self) -> List[TensorSpec]:
        specs = [TensorSpec(self.spec.embedding, (self.spec.vocab_size, self.spec.hidden_size), MATRIX)]
        if self.spec.position_table is not None:
            specs.append(TensorSpec(self.spec.position_table, (self.spec.max_positions, self.spec.hidden_size), MATRIX))
        for layer in self.layers:
            specs += layer.tensor_specs()
        for at, name in enumerate(self.spec.depth_weights or ()):
            specs.append(TensorSpec(name, (at + 2,), VECTOR, init=("normal", 1.0 / (at + 2), 0.02)))     # about an average
        specs += self._join_specs()
        specs += self.final_norm.tensor_specs()
        if self.spec.head is not None:
            specs.append(TensorSpec(self.spec.head, (self.spec.vocab_size, self.spec.hidden_size), MATRIX))
        return specs

    def _join_specs(self) -> List[TensorSpec]:
        join, hidden = self.spec.join, self.spec.hidden_size
        return [] if join is None else [TensorSpec(join.matrix, (hidden, 2 * hidden), MATRIX),
                                        TensorSpec(join.vectors, (len(join.before), hidden), VECTOR, init=("normal", 0.0, 0.02))]

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        tensors = dict(tensors)
        self.embedding = tensors.pop(self.spec.embedding).contiguous()
        if self.spec.position_table is not None:
            self.position_table = tensors.pop(self.spec.position_table).contiguous()
        self.head = tensors.pop(self.spec.head).contiguous() if self.spec.head is not None else self.embedding
        for layer in self.layers:
            layer.bind(tensors)
        if self.spec.depth_weights is not None:
            self.depth_weights = [tensors.pop(name).contiguous() for name in self.spec.depth_weights]
        if self.spec.join is not None:
            self.join_matrix = tensors.pop(self.spec.join.matrix).contiguous()
            # one tensor a pass: a row of the table need not begin where the kernels' 16-byte reads may
            self.join_vectors = [row.clone() for row in tensors.pop(self.spec.join.vectors)]
        self.final_norm.bind(tensors)
        for position in self.positions.values():
            position.prepare(self.spec.max_positions, self.device)

    # Auto: keep the second copies if they take at most this share of the device's memory and of what is free.
    STREAMED_SHARE_OF_DEVICE = 0.25
    STREAMED_SHARE_OF_FREE = 0.5

    def streamed_weights(self) -> List[torch.Tensor]:
        """Every matrix a decode step streams through ``ops.linear``: the layers' and the head."""
        found = [w for layer in self.layers if hasattr(layer, "streamed_weights") for w in layer.streamed_weights()]
        if self.join_matrix is not None:
            found.append(self.join_matrix)
        if self.head is not None:
            found.append(self.head)
        return found

    def keep_streamed_copies(self, wanted: Optional[bool] = None) -> int:
        """Keeps, beside every matrix that decode steps stream through, a second copy in the order in which
        the weight-streaming kernels read it fastest (``ops.tile_weight``; the row-major one stays for the
        library's products of prompt portions and for the token table).  The results are the same bit for
        bit; a decode step of few rows takes a sixth less time; the weights take twice the memory.
        ``wanted`` None decides by room: yes if the copies take at most a quarter of the device's memory
        and half of what is free.  Returns the bytes the copies take (0: none kept).  Asked again, it
        answers what it did the first time."""
        if self.streamed_copy_bytes is not None:
            return self.streamed_copy_bytes
        self.streamed_copy_bytes = 0
        weights = self.streamed_weights() if (self.dtype == torch.bfloat16 and wanted is not False) else []
        weights = [w for w in weights if w.is_cuda and w.dtype == torch.bfloat16 and w.dim() == 2 and w.shape[1] % 64 == 0]
        if not weights:
            return 0
        if wanted is None:
            needed = sum(-(-w.shape[0] // 16) * 16 * w.shape[1] * 2 for w in weights)
            free, total = torch.cuda.mem_get_info(weights[0].device)
            if needed > self.STREAMED_SHARE_OF_DEVICE * total or needed > self.STREAMED_SHARE_OF_FREE * free:
                return 0
        self.streamed_copy_bytes = sum(ops.keep_streamed_copy(w) for w in weights)
        return self.streamed_copy_bytes

    def row_tilings(self) -> list:
        """Every distinct tiling a part of the model declares, in a fixed order (``RowTiling``)."""
        found = []
        for layer in self.layers:
            for tiling in (layer.row_tilings() if hasattr(layer, "row_tilings") else []):
                if tiling is not None and tiling not in found:
                    found.append(tiling)
        return found

    # ---- bytes ---------------------------------------------------------------
    def weight_accounting(self, nbytes=None, rows: int = 1) -> Dict[str, object]:
        """Bytes of the model's tensors by class, as they lie in memory (``resident``) and as a decode step
        of ``rows`` rows reads them (``decode``): of the token table only the rows' own rows, and the whole
        table once more as the head if the head is tied to it (the reference's accounting,
        crates/leone/src/model.rs:306-366).  ``nbytes(spec)`` gives a tensor's size; by default its element
        count in this model's type."""
        size = 2 if self.dtype == torch.bfloat16 else 4
        if nbytes is None:
            def nbytes(spec):
                count = 1
                for extent in spec.shape:
                    count *= extent
                return count * size
        resident: Dict[str, int] = {"embed": 0, "head": 0}
        table = TensorSpec(self.spec.embedding, (self.spec.vocab_size, self.spec.hidden_size), MATRIX)
        resident["embed"] = nbytes(table)
        if self.spec.position_table is not None:
            resident["positions"] = nbytes(TensorSpec(self.spec.position_table, (self.spec.max_positions, self.spec.hidden_size), MATRIX))
        if self.spec.head is not None:
            resident["head"] = nbytes(TensorSpec(self.spec.head, (self.spec.vocab_size, self.spec.hidden_size), MATRIX))
        for layer in self.layers:
            for part in (layer.parts() if hasattr(layer, "parts") else (layer,)):
                family = getattr(part, "family", "layer")
                resident[family] = resident.get(family, 0) + sum(nbytes(s) for s in part.tensor_specs())
        resident["norm"] = resident.get("norm", 0) + sum(nbytes(s) for s in self.final_norm.tensor_specs())
        if self.spec.depth_weights is not None:
            resident["depth"] = sum(nbytes(TensorSpec(name, (at + 2,), VECTOR)) for at, name in enumerate(self.spec.depth_weights))
        if self.spec.join is not None:
            resident["join"] = sum(nbytes(s) for s in self._join_specs())
        decode = dict(resident)
        decode["embed"] = resident["embed"] // self.spec.vocab_size * rows
        if "positions" in decode:
            decode["positions"] = resident["positions"] // self.spec.max_positions * rows
        if self.spec.head is None:
            decode["head"] = resident["embed"]
        return {"tensor_bytes": sum(resident.values()), "resident": resident, "decode": decode,
                "streamed_copy_bytes": self.streamed_copy_bytes or 0}

    def weight_bytes(self) -> int:
        """Bytes of all tensors of the model."""
        return self.weight_accounting()["tensor_bytes"]

    def decode_step_weight_bytes(self, rows: int = 1) -> int:
        """Weight bytes a decode step of ``rows`` rows has to read: every weight it uses, once."""
        return sum(self.weight_accounting(rows=rows)["decode"].values())

    # ---- cache ---------------------------------------------------------------
    def cache_needs(self) -> Dict[int, object]:
        """Cache slot -> what the layer runs on it need (one need per slot).  A layer that needs several kinds
        of storage (``cache_need()`` answers with a dict, see ``parts.base.flatten_needs``) gets one slot for
        each, keyed (the run's slot, *names)."""
        needs: Dict[object, object] = {}
        writers: Dict[object, int] = {}
        for run in self.schedule:
            need = self.layers[run.layer].cache_need()
            leaves = flatten_needs(need)
            if not leaves:
                if run.cache is not None:
                    raise ValueError(f"layer {run.layer} keeps no cache but its run names slot {run.cache}")
                continue
            if run.cache is None:
                raise ValueError(f"layer {run.layer} needs a cache but its run names none")
            for path, leaf in leaves:
                lent = self._lender(run, need, path)
                key = ((run.cache if lent is None else lent,) + path) if isinstance(need, dict) else run.cache
                if key in needs and needs[key] != leaf:
                    raise ValueError(f"cache slot {key} is shared by layers with different needs")
                if lent is not None and key not in needs:
                    raise ValueError(f"layer {run.layer} borrows cache slot {key}, which no earlier run keeps")
                needs[key] = leaf
            writers[run.cache] = writers.get(run.cache, 0) + (1 if run.writes else 0)
        for slot, count in writers.items():
            if count != 1:
                raise ValueError(f"cache slot {slot} must have exactly one writing run, found {count}")
        return needs

    @staticmethod
    def _lender(run: LayerRun, need, path) -> Optional[int]:
        """The slot of the run that lends this run the storage at ``path`` of its needs, or None if it is its own."""
        if run.borrow and isinstance(need, dict) and path and path[0] in run.borrow:
            return run.borrow[path[0]]
        return None

    @staticmethod
    def _cache_of(run: LayerRun, layer, caches: Dict[object, CacheView]):
        """What a run's layer receives as its cache: the view of the run's slot, or, for a layer with several
        needs, the views in the shape of its needs."""
        if run.cache is None:
            return None

        def view(key, writes=run.writes):
            found = caches.get(key)
            if found is not None and found.writes != writes:
                found = type(found)(**{**found.__dict__, "writes": writes})
            return found

        need = layer.cache_need()
        if isinstance(need, dict):
            def lookup(key):
                lent = DecoderModel._lender(run, need, key[1:])
                return view(key, run.writes) if lent is None else view((lent,) + key[1:], False)
            return nest_views(need, (run.cache,), lookup)
        return view(run.cache)

    def _mix_depth(self, x: torch.Tensor, pending, history: torch.Tensor, at: int):
        """x + pending is run ``at``'s own result: it is kept, and the stream becomes the weighted sum of all results
        so far, in one kernel."""
        scale = 1.0
        if isinstance(pending, ops.PreparedRows):
            pending = None
        elif isinstance(pending, ops.ScaledDelta):
            pending, scale = pending.rows, pending.scale
        elif isinstance(pending, (ops.NormedDelta, ops.MixedDelta)):
            pending = pending.materialize()
        ops.depth_mix(x, pending, scale, history, at + 2, self.depth_weights[at])
        return None

    def _join_stream(self, x: torch.Tensor, pending, first: torch.Tensor, t: int, step: StepContext):
        """The stream with what is pending goes into the operand of the joining product beside ``first`` and becomes the pass's
        vector; what comes back is that product, still to be added."""
        operand = ops.stream_join(x, ops.delta_terms(pending), first, self.join_vectors[t], step.dtype)
        return ops.linear(operand, self.join_matrix, out_dtype=torch.float32, planes_ok=True)

    # ---- forward ---------------------------------------------------------------
    def forward(self, tokens: torch.Tensor, step: StepContext, caches: Dict[int, CacheView]) -> Optional[torch.Tensor]:
        """Runs the step's rows through every scheduled layer; returns float32 logits of the wanted rows."""
        if self.position_table is not None and step.max_position >= self.position_table.shape[0]:
            raise ValueError(f"position {step.max_position} is beyond the position table of {self.position_table.shape[0]} rows")
        first = None
        if self.joins:                        # the embedding's output is asked for again: the embedding writes it twice
            first = torch.empty((tokens.numel(), self.spec.hidden_size), dtype=torch.float32, device=tokens.device)
        x = ops.embed(self.embedding, tokens, scale=1.0 if self.spec.embedding_scale is None else self.spec.embedding_scale,
                      position_table=self.position_table, positions=step.positions, copy=first)
        pending = None
        history = None
        if self.depth_weights is not None:
            # every run's own result is kept for the step: the stream behind a run is mixed from all of them
            history = torch.empty((len(self.schedule) + 1, *x.shape), dtype=torch.float32, device=x.device)
            history[0].copy_(x)
        for at, run in enumerate(self.schedule):
            layer = self.layers[run.layer]
            cache = self._cache_of(run, layer, caches)
            if at in self.joins:
                pending = self._join_stream(x, pending, first, self.joins[at], step)
            # A block that can do so leaves the first norm of the block that runs next prepared.
            after = self.layers[self.schedule[at + 1].layer] if at + 1 < len(self.schedule) and at + 1 not in self.joins else None
            next_norm = after.entry_norm(step.dtype) if hasattr(after, "entry_norm") else None
            if next_norm is not None and getattr(layer, "prepares_next", False):
                pending = layer.forward(x, pending, step, cache, next_norm=next_norm)
            else:
                pending = layer.forward(x, pending, step, cache)
            if history is not None:
                pending = self._mix_depth(x, pending, history, at)
        if step.want_rows is None or step.want_rows.numel() == 0:
            if pending is not None:
                pass  # nothing reads the last delta when no logits are wanted
            return None
        if isinstance(pending, ops.PreparedRows):
            pending = None                    # prepared for a norm that never ran: the stream is up to date
        if isinstance(pending, (ops.ScaledDelta, ops.MixedDelta)) and not hasattr(self.final_norm, "gain"):
            pending = pending.materialize()
        if hasattr(self.final_norm, "lazy"):
            y = self.final_norm.lazy(x, pending, self.dtype, rows=step.want_rows)
        else:
            y = self.final_norm.add_norm(x, pending, self.dtype, rows=step.want_rows)
        logits = ops.linear(y, self.head, out_dtype=torch.float32)
        return ops.soft_cap(logits, self.spec.logit_cap) if self.spec.logit_cap else logits
