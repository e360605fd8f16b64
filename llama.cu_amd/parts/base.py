"""What a model is made of: specifications (data), parts (objects that hold weights
and run kernels) and the registries that turn the first into the second.

A *specification* is plain data: a kind, parameters, and the name under which the
part's tensors lie in the weight file.  A *part* is built from a specification by
the registry of its category:

  ``norm``      ``forward(x, delta) -> y``             x: float32 [n, d] residual stream, updated in
                                                    place by ``x += delta`` (``delta`` may be None);
                                                    y: [n, d] in the compute type
  ``mixer``     ``forward(h, step, cache) -> delta``   h, delta: [n, d] compute type; ``step`` is the
                ``cache_need() -> need or None``       batch (engine.batch.StepContext); ``cache`` is
                                                    what the engine made for ``cache_need()``
  ``ffn``       ``forward(h) -> delta``
  ``position``  ``tables(...)``/``apply(...)``         see parts.position
  ``block``     ``forward(x, pending, step, cache) -> pending``   the arrangement of the four above
  ``stream``    ``forward(x, pending, start) -> x``     a change of the residual stream between two layers; ``start`` is what
                ``begin(x)`` made of the embedding's output

Every part also has ``tensors() -> {relative name: TensorSpec}``,
``load(tensors, build)`` and the flag ``graph_safe`` (see Part).  No part knows which model it is in: sizes and constants
arrive as parameters.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Callable, Dict, List, Optional, Tuple

import torch


@dataclass(frozen=True)
class TensorSpec:
    """One tensor a part binds: its shape, and how a random model fills it: the name of an
    initialiser (``normal``: N(0, std); ``one_plus_normal``: 1 + N(0, std), for norm weights;
    ``identity_plus_normal``; ``zeros``; ``ones``; or one that ``weights.register_initialiser`` has made known).
    ``integer`` tensors are kept as int32, all others follow the weight policy."""
    shape: Tuple[int, ...]
    init: str = "normal"
    integer: bool = False
    optional: bool = False        # a file may lack it
    random: bool = True           # the random-weights mode makes it


@dataclass
class PartSpec:
    kind: str
    params: Dict[str, Any] = field(default_factory=dict)
    name: str = ""           # the part's component in tensor names ("self_attn", "mlp", ...)


@dataclass(frozen=True)
class RunEntry:
    """One step of the run order: which layer runs, and whose cache it uses.  ``cache_of``
    None: a cache of its own.  ``cache_of = j``: it reads the cache that entry ``j`` of the
    run order wrote (and writes none).  ``before = k``: the residual stream passes the model's stream
    part ``k`` (``ModelSpec.streams``) right before the layer runs."""
    layer: int
    cache_of: Optional[int] = None
    before: Optional[int] = None


@dataclass
class ModelSpec:
    """A whole decoder as data."""
    hidden_size: int
    vocab_size: int
    max_positions: int
    embedding: PartSpec
    layers: List[PartSpec]              # block specifications, each with its tensor-name prefix
    run_order: List[RunEntry]
    final_norm: PartSpec
    head: PartSpec
    eos_token_ids: Tuple[int, ...] = ()
    streams: List[PartSpec] = field(default_factory=list)    # changes of the stream that entries of the run order name


# ------------------------------------------------------------------ cache needs


@dataclass
class LayerCache:
    """What one entry of the run order gets: the pages of its layer (``pages``,
    ``[num_pages, 2, kv_heads * head_dim * page_size]``) with the group whose block tables
    index them, whether the entry writes them, and/or its per-request state
    (``state``, ``[slots, *shape]``)."""
    group: int = -1
    pages: Optional[torch.Tensor] = None
    writes: bool = True
    state: Optional[torch.Tensor] = None
    page_size: int = 0          # tokens per page of ``pages`` (0: no pages)
    more: Dict[str, torch.Tensor] = field(default_factory=dict)   # the block's own states by name (``Part.own_states``)


class CacheNeed:
    """What a mixer asks of the cache manager.  The engine knows no kind of need by name: it asks
    every need these questions.

    ``pool()``        None, or ``(window, page_size)``: the need is pages of keys and values, and needs
                      with an equal answer share one pool of page ids and one block table per request
                      (``window`` 0: every token is kept; w: pages that a window of w tokens has
                      passed are given back; ``page_size`` 0: the engine's default);
    ``page_bytes(page_size, elem_size)``   bytes of one page of this need (0 if it has no pages);
    ``allocate(group, num_pages, page_size, slots, dtype, device)``   the memory, as a LayerCache;
    ``can_truncate``  whether what the need holds for a request can be cut back to a shorter
                      length (pages can; a state that has folded tokens in cannot).  A request
                      whose cache cannot be cut back and has to be (an end-of-sequence token
                      learned after more was computed) loses its cache and is computed again from
                      its tokens when it goes on.
    """
    can_truncate = True

    def pool(self):
        return None

    def page_bytes(self, page_size: int, elem_size: int) -> int:
        return 0

    def allocate(self, group: int, num_pages: int, page_size: int, slots: int, dtype, device) -> LayerCache:
        return LayerCache()


@dataclass(frozen=True)
class PagedKV(CacheNeed):
    """Keys and values of every token (or of the last ``window`` tokens), in pages.  ``value_dim``: the values'
    head size if it is not the keys' (a page then holds all its keys, then all its values, in one row)."""
    kv_heads: int
    head_dim: int
    window: int = 0          # 0: all tokens
    page_size: int = 0       # tokens per page; 0: the engine's default
    value_dim: int = 0       # 0: head_dim

    def pool(self):
        return (self.window, self.page_size)

    def page_bytes(self, page_size: int, elem_size: int) -> int:
        return self.kv_heads * (self.head_dim + (self.value_dim or self.head_dim)) * page_size * elem_size

    def allocate(self, group, num_pages, page_size, slots, dtype, device) -> LayerCache:
        if self.value_dim and self.value_dim != self.head_dim:
            shape = (num_pages, 1, self.kv_heads * (self.head_dim + self.value_dim) * page_size)
        else:
            shape = (num_pages, 2, self.kv_heads * self.head_dim * page_size)
        return LayerCache(group=group, pages=torch.zeros(shape, dtype=dtype, device=device), page_size=page_size)


@dataclass(frozen=True)
class SlotState(CacheNeed):
    """A state of fixed size per request (``shape`` without the slot axis).  The mixer that owns
    it starts it anew when a request's first token (position 0) comes."""
    shape: Tuple[int, ...]
    dtype: torch.dtype = torch.float32
    can_truncate = False

    def allocate(self, group, num_pages, page_size, slots, dtype, device) -> LayerCache:
        return LayerCache(state=torch.zeros((slots,) + tuple(self.shape), dtype=self.dtype, device=device))


@dataclass(frozen=True)
class SeveralNeeds(CacheNeed):
    """The needs of a mixer that is several mixers side by side, each with a need of its own: at most one of them
    pages (its pool is the whole's), the others states of fixed size.  The mixers all get the one LayerCache: the
    pages in ``pages``, a single state in ``state``, and with more than one state the i-th need's as
    ``more["state<i>"]`` (``state`` is then the first)."""
    needs: Tuple[CacheNeed, ...]

    def __post_init__(self):
        if sum(1 for n in self.needs if n.pool() is not None) > 1:
            raise ValueError("several needs side by side: at most one of them may be pages of keys and values")

    @property
    def can_truncate(self):
        return all(n.can_truncate for n in self.needs)

    def pool(self):
        for n in self.needs:
            if n.pool() is not None:
                return n.pool()
        return None

    def page_bytes(self, page_size: int, elem_size: int) -> int:
        return sum(n.page_bytes(page_size, elem_size) for n in self.needs)

    def allocate(self, group, num_pages, page_size, slots, dtype, device) -> LayerCache:
        out = LayerCache()
        states = 0
        for i, n in enumerate(self.needs):
            made = n.allocate(group, num_pages, page_size, slots, dtype, device)
            if made.pages is not None:
                out.group, out.pages, out.page_size = made.group, made.pages, made.page_size
            if made.state is not None:
                if out.state is None:
                    out.state = made.state
                out.more[f"state{i}"] = made.state
                states += 1
        return out


# ------------------------------------------------------------------ building


@dataclass
class BuildContext:
    """What a part may need to know about the engine while it binds its weights."""
    dtype: torch.dtype               # the compute type: torch.bfloat16 or torch.float32
    device: torch.device
    max_positions: int
    page_size: int
    pack_weights: bool = True        # keep a second copy of bfloat16 matrices in the order the decode kernel streams them


@dataclass
class ScaledRows:
    """Rows on their way from a norm to a matrix product whose normalisation is still to be
    applied: the norm's weight is in already, and row ``i`` of whatever is multiplied with
    them is to be multiplied by ``rsqrt(sum(sumsq[i]) / width + eps)``.  A mixer that can end
    with the residual sum and the next norm's weight in its last product hands these to a
    feed-forward that can apply the factor in its first product's epilogue, and no norm
    kernel runs between them.  A part that does not know of this never sees one: the block
    offers it only to parts that say they take it."""
    rows: torch.Tensor          # [n, width], the compute type
    sumsq: torch.Tensor         # [n, parts] float32 shares of the rows' sums of squares
    width: int
    eps: float


@dataclass
class NormedRows:
    """The rows that a block's first norm would make of the residual stream, made already by the block before (in
    the kernel that added that block's last output to the stream): ``rows [n, width]`` in the compute type.  A
    block hands these only to a block that says it takes them (``takes_normed_rows``)."""
    rows: torch.Tensor


@dataclass
class StreamUpdate:
    """A sublayer's output on its way into several residual streams (``parts/streams.py``): ``x_t <- sum_s mix[s, t] x_s + out[t] *
    delta``, all streams at once.  Whoever norms next lets it in."""
    delta: torch.Tensor         # [n, width] in the compute type or float32, or float32 planes [planes, n, width]
    mix: torch.Tensor           # [streams, streams] float32: from, to
    out: torch.Tensor           # [streams] float32

    def at_rows(self, gather) -> "StreamUpdate":
        return StreamUpdate(gather(self.delta), self.mix, self.out)


@dataclass
class StreamsEnd:
    """What ``forward(..., into=)`` of a branch takes instead of ``(residual, norm)`` where there are several residual streams: the
    branch's last product may let its output into them (``mix``, ``out`` as in ``StreamUpdate``) and return ScaledRows made with
    ``norm`` of the sum of the streams weighted with ``read`` (None: ones)."""
    x: torch.Tensor
    norm: Any                   # parts.streams.StreamsNorm
    read: Optional[torch.Tensor]
    mix: torch.Tensor
    out: torch.Tensor


class Part:
    # Whether a step through this part may be captured into a graph and replayed: true only
    # if all it does is launch work on the current stream whose shape depends on the batch's
    # sizes alone, never on values it reads on the host (lengths, positions, slots).
    graph_safe = False

    # ---- what a part may offer so that kernels between it and its neighbours are saved.  All of it is
    # optional: a part that leaves these as they are is never given anything but plain rows, and
    # everything it returns is plain rows; blocks and the model ask through these names only.
    #
    # norm:  ``deferrable``: the norm is a factor per row times a weight per column (``weight``, ``size``,
    #        ``eps``), so the factor may be applied after the next matrix product (ScaledRows);
    #        ``takes_planes``: ``forward(x, delta)`` also takes float32 planes ``[planes, rows, width]``
    #        of partial sums as ``delta``;
    #        ``delta_scale``: what ``delta`` is multiplied by before it is added to the stream, also by a
    #        product that ends in this norm.
    # mixer, feed-forward:  ``ends_in_norm``: ``forward(..., into=(residual, norm))`` (or a StreamsEnd) may add its output to
    #        the residual stream itself and return ScaledRows made with ``norm``;
    #        ``ends_in_planes``: ``forward(..., planes_ok=True)`` may return float32 planes;
    #        ``takes_scaled_rows(n_rows)``: whether ``forward`` takes ScaledRows of that many rows;
    #        ``reads_float32``: a mixer whose rows go on in 32-bit: the block's norm writes float32 rows for it.
    # block: ``ends_in_next_norm``: ``forward(..., next_norm=)`` may end in the norm that follows the block;
    #        ``ends_in_planes`` / ``takes_planes`` / ``takes_scaled_rows`` as above, for its last branch
    #        and its first norm.
    #        ``hands_over_normed``: ``forward(..., next_norm=)`` adds its last output to the stream itself, runs that
    #        norm in the same kernel and returns NormedRows; ``takes_normed_rows``: ``pending`` may be NormedRows
    #        made with its ``first_norm``.
    deferrable = False
    delta_scale = 1.0
    reads_float32 = False
    # embedding, block, final norm: how many residual streams a row holds side by side (all three agree)
    streams = 1
    # mixer: ``splits_output``: its last step is a product with ``output_matrix`` ([width, output_width], known after ``load``), and
    # ``forward_rows(h, step, cache, out, factor, state=)`` writes what it would multiply, times ``factor``, into the columns ``out``
    # instead: several such mixers' rows side by side are one product.  ``own_output`` False (set before ``load``): somebody else
    # multiplies, so the part keeps no matrix of its own for it.
    splits_output = False
    own_output = True
    takes_planes = False
    ends_in_norm = False
    ends_in_planes = False
    ends_in_next_norm = False
    hands_over_normed = False
    takes_normed_rows = False

    def takes_scaled_rows(self, n_rows: int) -> bool:
        return False

    # block: the norm that a block starts with, if whoever runs before it may end in it (else None)
    first_norm = None

    def decode_splits(self, batch: int, max_ctx_len: int) -> int:
        """Into how many parts a mixer (or a block, for its mixer) wants a decoding request's keys cut when
        ``batch`` requests decode over at most ``max_ctx_len`` keys; a captured graph fixes the number."""
        return 1

    # position: what a position encoding may be, each optional (``parts/position.py`` describes them): tables of
    # a rotation, any other change of queries and keys in place, a bias inside the scores.
    def rotary_tables(self):
        return None

    def rotated_dims(self) -> int:
        """position: how many dims of a head a rotation turns (0: none); known before the tables are made."""
        return 0

    def apply(self, qkv, positions, heads, kv_heads, head_dim) -> None:
        pass

    def score_slopes(self):
        return None

    def tensors(self) -> Dict[str, TensorSpec]:
        return {}

    def load(self, tensors: Dict[str, torch.Tensor], build: BuildContext) -> None:
        pass

    def own_states(self) -> Dict[str, "SlotState"]:
        """block: states of fixed size per request that the block itself keeps, beside what its mixer asks for with
        ``cache_need`` (the last inputs of a convolution over time, say), by name.  Every entry of the run order
        gets its own, also one that reads another entry's keys and values; ``forward`` finds them in
        ``cache.more[name]`` as ``[slots, *shape]``.  Like any SlotState they are not cleared when a slot changes
        hands: their owner starts them anew at a request's position 0."""
        return {}

    def prepare(self, step) -> None:
        """Called once per step for every layer, on the host, before the step's arrays go to the device and
        before anything of the step runs or is replayed from a graph: a part that derives arrays from the batch
        (lists of tasks, orders) writes them into ``step.extra(name, size)`` here, so that its ``forward`` launches
        work whose shape depends on the step's sizes alone and a graph-safe part stays one."""
        pass

    def fused_groups(self, dtype: torch.dtype, device: torch.device) -> List[Tuple[Tuple[str, ...], int]]:
        """Tensors that this part multiplies as one matrix: ``[(names in row order, rows to which each
        is filled up with zeros, or 0)]``.  The weight loader lays such tensors out one after the other,
        so that the part finds the fused matrix in place (``weights.loader.fused_rows``)."""
        return []


_REGISTRIES: Dict[str, Dict[str, Callable[..., Part]]] = {
    "norm": {}, "mixer": {}, "ffn": {}, "position": {}, "block": {}, "embedding": {}, "head": {},
    "stream": {}}


def register_part(category: str, kind: str, factory: Callable[..., Part], replace: bool = False) -> None:
    """Make ``kind`` known in ``category``; ``factory(**params)`` builds the part."""
    reg = _REGISTRIES.get(category)
    if reg is None:
        raise ValueError(f"no part category {category!r}; categories: {sorted(_REGISTRIES)}")
    if kind in reg and not replace:
        raise ValueError(f"{category} part {kind!r} is already registered")
    reg[kind] = factory


def make_part(category: str, spec: PartSpec) -> Part:
    reg = _REGISTRIES[category]
    factory = reg.get(spec.kind)
    if factory is None:
        raise ValueError(f"no {category} part of kind {spec.kind!r}; registered: {sorted(reg)}")
    return factory(**spec.params)


def registered_parts(category: str) -> List[str]:
    return sorted(_REGISTRIES[category])


def prefixed(prefix: str, name: str) -> str:
    return f"{prefix}.{name}" if prefix else name
