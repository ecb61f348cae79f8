"""Interfaces of the parts a layer is made of, and the registries that build them.

A part is built from a `PartSpec` (its sizes and constants) and the activation dtype; it
declares the tensors it needs under a name prefix, loads them from a weight store, and
runs on the tokens of one step.  A part never learns which model it is in.

  Mixer            forward(x, ctx, cache) -> y        x, y: [T, hidden]; y may also be a stack
                                                      [P, T, hidden] of float32 partial sums,
                                                      which the next norm adds in order
                   cache_need() -> KVNeed | None      paged keys/values it wants
                   state_need() -> StateNeed | None   fixed-size per-request state it wants
  FeedForward      forward(x, ctx) -> y               (y as for the mixer)
  Norm             forward(resid, add, out_dtype, rows=None, out=None) -> normed
                   resid is the float32 residual stream; `add` (if given) is summed into
                   it first; with `rows` only those rows are produced and resid is not
                   changed.  A kind that can add `add_scale * add` takes that keyword too
                   (it is only passed where the factor is not 1).
                   forward_branch(resid, y, rows_dtype): resid += norm(y), for blocks that norm
                   a sublayer's output instead of its input.
  PositionEncoding data for the mixer's fused kernel (for "rope": cos/sin tables)
  Block            forward(stream, ctx, cache) -> stream, the arrangement of the above
                   around the residual stream.
  TokenEmbedding   forward(ids, ctx) -> float32 [T, hidden], the start of the residual stream
                   (`ctx` for kinds that need positions or the request; the built-in one
                   ignores it); `table` is what a tied head shares
  Head             forward(h) -> float32 logits [R, vocab]; load(..., shared=) takes the
                   embedding's table when the spec says `tied`
  StreamOp         forward(stream, first, ctx) -> stream: a change of the stream between two runs
                   of layers (what a pass over a span of layers adds when it starts, what a layer
                   adds behind its branches, an average over the layers so far)

New kinds register themselves with the decorators below; a `PartSpec.kind` then selects
them.  Nothing else in the engine has to change.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Callable, Dict, List, Optional, Sequence, Tuple

import torch

from ..config.spec import LayerSpec, PartSpec
from ..weights.store import TensorDecl, WeightStore


# ---- what a layer may ask of the cache ------------------------------------------------
PAGE = -1      # in a pool's shape: the axis that is as long as a page has tokens
PAGE_BY_8 = -8 # the axis that is an eighth of that (-n: the page's tokens divided by n, which must divide them)


@dataclass(frozen=True)
class PoolNeed:
    """One paged pool of a layer: the runner allocates [pages, *shape] with PAGE replaced by the
    page size (PAGE_BY_8: by an eighth of it), in `dtype` (None: the activation dtype), and hands it to
    the mixer under `name`.  A shape has one such axis."""
    name: str
    shape: Tuple[int, ...]
    dtype: Optional[torch.dtype] = None

    def bytes_per_token(self, element_size: int) -> int:
        n, by = 1, 1
        for s in self.shape:
            if s < 0:
                by = -int(s)
            else:
                n *= int(s)
        return n // by * (element_size if self.dtype is None else torch.tensor([], dtype=self.dtype).element_size())


@dataclass(frozen=True)
class KVNeed:
    """What a mixer keeps in pages: `window` = 0 keeps every token's entry, w > 0 the last w (pages
    that the window has passed go back to the pool while the request runs); `pools` names the
    pools and the shape of a page in each.  `KVNeed.keys_values` is the pair that attention keeps;
    a mixer of another kind may keep one pool (a latent), or pools of different widths."""
    window: int = 0
    pools: Tuple[PoolNeed, ...] = ()

    @staticmethod
    def keys_values(num_kv_heads: int, head_dim: int, window: int = 0, v_grouped: bool = False,
                    value_dim: Optional[int] = None) -> "KVNeed":
        """K pool "k" [pages, kv_heads, page_size, head_dim]; V pool "v" [pages, kv_heads, page_size, value_dim]
        (`value_dim`: head_dim unless given), or with `v_grouped` [pages, kv_heads, page_size / 8, value_dim, 8]
        (eight keys side by side for every dim)."""
        dv = head_dim if value_dim is None else int(value_dim)
        k = PoolNeed("k", (num_kv_heads, PAGE, head_dim))
        v = PoolNeed("v", (num_kv_heads, PAGE_BY_8, dv, 8) if v_grouped else (num_kv_heads, PAGE, dv))
        return KVNeed(window, (k, v))


@dataclass(frozen=True)
class StateNeed:
    """Fixed-size state per live request: one slot of this shape and dtype.  A part that keeps several (a
    matrix and the last inputs of a convolution, say) returns a tuple of them from `state_need`, each with a
    `name` of its own; the first is `LayerCache.state`, all are in `LayerCache.states` by name."""
    shape: Tuple[int, ...]
    dtype: torch.dtype = torch.float32
    name: str = "state"


def state_needs_of(need) -> Tuple["StateNeed", ...]:
    """What `state_need()` returned (None, one StateNeed, or several) as a tuple with names of their own."""
    if need is None:
        return ()
    needs = (need,) if isinstance(need, StateNeed) else tuple(need)
    if len({n.name for n in needs}) != len(needs):
        raise ValueError("the states of one part need names of their own")
    return needs


@dataclass
class LayerCache:
    """What one run of a layer gets from the cache.  `write` is False when the run reads
    the cache that another layer's run owns."""
    group: int = -1
    pools: Dict[str, torch.Tensor] = field(default_factory=dict)   # by PoolNeed.name: [pages, *shape]
    state: Optional[torch.Tensor] = None      # [max_requests, *StateNeed.shape] (the first, if the part keeps several)
    write: bool = True
    states: Dict[str, torch.Tensor] = field(default_factory=dict)   # by StateNeed.name

    @property
    def k(self) -> Optional[torch.Tensor]:
        return self.pools.get("k")

    @property
    def v(self) -> Optional[torch.Tensor]:
        return self.pools.get("v")


@dataclass
class StepContext:
    """Everything about one step's batch that parts may read.  Device tensors unless
    marked host."""
    num_tokens: int
    num_seqs: int
    dtype: torch.dtype                         # activation dtype
    device: torch.device
    positions: torch.Tensor                    # int32 [T]   absolute position of each token
    tok_seq: torch.Tensor                      # int32 [T]   row of the batch each token is in
    cu_q: torch.Tensor                         # int32 [B+1] token offsets of the sequences
    ctx_lens: torch.Tensor                     # int32 [B]   cached length after this step
    state_slots: torch.Tensor                  # int64 [B]   per-request state slot
    slots: List[torch.Tensor]                  # per group int64 [T] cache slot of each token
    block_tables: List[torch.Tensor]           # per group int32 [B, max_pages]
    cu_q_host: Sequence[int] = ()              # host copies for choosing kernels
    ctx_lens_host: Sequence[int] = ()
    max_q_len: int = 0
    max_ctx_len: int = 0
    similar_lengths: bool = False              # host: the mean cached length is at least 0.9 of the longest
    no_slots: Optional[torch.Tensor] = None    # int64 [T] of -1: "store nothing"
    empty_f32: Optional[torch.Tensor] = None   # float32 [1, 0]: tables of "no rotation"
    scratch: Dict[Any, Any] = field(default_factory=dict)   # per-step data that kernels derive once
    ids: Optional[torch.Tensor] = None         # int32 [T]   the step's token ids (set by the model)


@dataclass
class NormSink:
    """Given to the part that runs before a norm: "add your result into `resid` yourself and
    prepare `norm`'s input".  A part that can (its last product, for few rows) answers with a
    `Folded`; it may always answer with its plain result instead."""
    resid: torch.Tensor                        # float32 [T, H], the residual stream
    norm: "Norm"


@dataclass
class Folded:
    """Rows whose norm is half done by the product before it: the stream already holds the sum,
    `xg` = round(stream * norm.weight) [T, H], `ss` [T, parts] float32 the parts of each row's
    sum of squares.  The product after the norm takes it in place of normed rows and scales its
    own rows by rsqrt(sum(ss) / H + eps) (`kernels.linear_fold_in`)."""
    xg: torch.Tensor
    ss: torch.Tensor
    norm: "Norm"

    def rows(self, dtype: torch.dtype) -> torch.Tensor:
        """The normed rows themselves, for a consumer without the folded product."""
        inv = torch.rsqrt(self.ss.sum(dim=1) / self.xg.shape[1] + self.norm.eps)
        return (self.xg.float() * inv[:, None]).to(dtype)


@dataclass
class Term:
    """Something the stream is to get: scale * y, or with a `weight` (float32 [H]) scale * (y / sqrt(mean(y^2) + eps)) *
    weight (with `groups`: in that many equal parts of the row, each divided by its own root mean square).  y: rows in either precision, or a stack [P, T, H] of float32 partial sums."""
    y: torch.Tensor
    weight: Optional[torch.Tensor] = None
    eps: float = 0.0
    scale: float = 1.0
    groups: int = 1


@dataclass
class DepthAverage:
    """What is to become of the stream once its terms are added: the sum s is the `place`-th result of the layers (kept in
    `results` [N, T, H], after the `place` results before it), and the stream becomes weights[0] first + sum over the results
    before of weights[1 + j] results[j] + weights[place + 1] s (`first`: the embedding's output)."""
    first: torch.Tensor
    results: torch.Tensor
    place: int
    weights: torch.Tensor


@dataclass
class Stream:
    """The residual stream between blocks: `resid` float32 [T, H], and a branch output
    `pending` that has not been added to it yet (the next norm adds it in the same
    kernel that norms), or `folded`: the branch output is already added and the next
    norm (`folded.norm`) half done.  A stream with `terms` or an `average` is `open`: who reads it next
    adds them (`parts.joining.join`, which can norm the new rows in the same pass); parts that know
    nothing of it are given a joined one."""
    resid: torch.Tensor
    pending: Optional[torch.Tensor] = None
    folded: Optional[Folded] = None
    rows: Optional[torch.Tensor] = None       # `resid` rounded to the activation dtype, as it is now (nothing
                                              # pending): what a sublayer that reads the stream itself takes
    pending_scale: float = 1.0                # the stream is to get pending_scale * pending
    terms: Tuple[Term, ...] = ()              # what it is to get besides
    average: Optional[DepthAverage] = None    # and what is then to become of it

    @property
    def open(self) -> bool:
        return bool(self.terms) or self.average is not None


class Part:
    # True if `forward` reads nothing of the step on the host (no lengths, no device-to-host
    # copies) and launches the same kernels for every step of the same batch size, so that a
    # decode step can be recorded once as a HIP graph and replayed.  Parts that do not say so
    # keep the whole model on the launch-by-launch path.
    graph_safe = False
    # Folding a norm into the products around it (see `Folded`): a mixer or feed-forward whose
    # `forward` takes a keyword `sink: Optional[NormSink]` says `takes_sink`; one whose `forward`
    # takes a `Folded` in place of its input rows says `takes_folded`; a norm that can be folded
    # (a weight vector `weight` in float32, `eps`, `dim`) says `foldable`.  One that the pass over an open stream can make
    # (the same, over `groups` equal parts of the row) says `joinable`.
    takes_sink = False
    takes_folded = False
    foldable = False
    joinable = False

    def __init__(self, spec: PartSpec, dtype: torch.dtype):
        self.spec = spec
        self.dtype = dtype

    @classmethod
    def declare(cls, spec: PartSpec, prefix: str) -> List[TensorDecl]:
        return []

    def load(self, store: WeightStore, prefix: str, device) -> None:
        pass


class Mixer(Part):
    def cache_need(self) -> Optional[KVNeed]:
        return None

    def state_need(self) -> Optional[StateNeed]:
        return None

    def forward(self, x: torch.Tensor, ctx: StepContext, cache: LayerCache) -> torch.Tensor:
        raise NotImplementedError

    def forward_terms(self, x: torch.Tensor, ctx: StepContext, cache: LayerCache) -> Tuple["Term", ...]:
        """The result as terms whose sum it is, for blocks that add them in a pass of their own; a mixer that ends in
        a sum of (normed) branches can hand those on."""
        return (Term(self.forward(x, ctx, cache)),)


class FeedForward(Part):
    def forward(self, x: torch.Tensor, ctx: StepContext) -> torch.Tensor:
        raise NotImplementedError


class Norm(Part):
    def forward(self, resid: torch.Tensor, add: Optional[torch.Tensor], out_dtype: torch.dtype,
                rows: Optional[torch.Tensor] = None, out: Optional[torch.Tensor] = None) -> torch.Tensor:
        raise NotImplementedError

    def forward_branch(self, resid: torch.Tensor, y: torch.Tensor, rows_dtype: Optional[torch.dtype]) -> Optional[torch.Tensor]:
        """The norm of a branch's OUTPUT, added into the stream: resid += norm(y) in place (y rows, or a
        stack [P, T, H] of float32 partial sums); returns the new resid rounded to `rows_dtype` (None: nothing).
        For arrangements whose sublayers read the stream itself ("branchnorm"); a norm kind that is only
        ever used before a sublayer need not have it."""
        raise NotImplementedError(f"norm kind {getattr(self, 'kind', type(self).__name__)!r} cannot norm a branch's output")


class PositionEncoding(Part):
    """What a mixer reads of it is between the two.  The built-in attention mixer reads a
    rotation: `cos` and `sin`, float32 tables [max_positions, rotary_dim / 2] on the device
    (made in `load`), `rotary_dim` (even, at most the head size) and `interleaved` (pairs
    (2i, 2i+1) instead of (i, i + rotary_dim / 2)); its kernels apply them to q and k."""


class TokenEmbedding(Part):
    table: Optional[torch.Tensor] = None

    def state_need(self) -> Optional[StateNeed]:
        """Fixed-size state per live request that the embedding itself keeps (the token before, say); a kind that
        returns one gets `forward(ids, ctx, cache=LayerCache)` with its slots."""
        return None

    def forward(self, ids: torch.Tensor, ctx: StepContext) -> torch.Tensor:
        raise NotImplementedError


class StreamOp(Part):
    """Something that changes the residual stream between two runs of layers (`ScheduleEntry.before` and `after`):
    forward(stream, first, ctx) -> stream, with `first` the embedding's output as it was before the first layer
    (float32 [T, H]; None unless the kind says `needs_first`)."""
    needs_first = False
    writes_stream = True       # `forward` may change the stream's tensor in place
    takes_open = False         # `forward` takes a stream that is `open`

    def forward(self, stream: "Stream", first: Optional[torch.Tensor], ctx: StepContext) -> "Stream":
        raise NotImplementedError


class Head(Part):
    tied = False

    def load(self, store: WeightStore, prefix: str, device, shared: Optional[torch.Tensor] = None) -> None:
        raise NotImplementedError

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        raise NotImplementedError


class Block:
    """Arrangement of a layer's parts around the residual stream."""

    graph_safe = False
    writes_stream = True       # `forward` may change the stream's tensor in place
    takes_open = False         # `forward` takes a stream that is `open` (see `Stream`)

    def __init__(self, layer: LayerSpec, dtype: torch.dtype):
        self.layer = layer
        self.dtype = dtype

    @classmethod
    def declare(cls, layer: LayerSpec) -> List[TensorDecl]:
        raise NotImplementedError

    def load(self, store: WeightStore, device) -> None:
        raise NotImplementedError

    def cache_need(self) -> Optional[KVNeed]:
        return None

    def state_need(self) -> Optional[StateNeed]:
        return None

    def forward(self, stream: Stream, ctx: StepContext, cache: LayerCache) -> Stream:
        raise NotImplementedError


# ---- registries -------------------------------------------------------------------------
MIXERS: Dict[str, type] = {}
FEED_FORWARDS: Dict[str, type] = {}
NORMS: Dict[str, type] = {}
POSITION_ENCODINGS: Dict[str, type] = {}
BLOCKS: Dict[str, type] = {}
EMBEDDINGS: Dict[str, type] = {}
HEADS: Dict[str, type] = {}
STREAM_OPS: Dict[str, type] = {}


def _register(table: Dict[str, type], what: str) -> Callable[[str], Callable[[type], type]]:
    def named(kind: str) -> Callable[[type], type]:
        def deco(cls: type) -> type:
            table[kind] = cls
            cls.kind = kind
            return cls
        return deco
    return named


register_mixer = _register(MIXERS, "mixer")
register_feed_forward = _register(FEED_FORWARDS, "feed-forward")
register_norm = _register(NORMS, "norm")
register_position_encoding = _register(POSITION_ENCODINGS, "position encoding")
register_block = _register(BLOCKS, "block")
register_embedding = _register(EMBEDDINGS, "embedding")
register_head = _register(HEADS, "head")
register_stream_op = _register(STREAM_OPS, "stream op")


def _lookup(table: Dict[str, type], what: str, kind: str) -> type:
    try:
        return table[kind]
    except KeyError:
        raise KeyError(f"unknown {what} kind {kind!r} (registered: {', '.join(sorted(table))})") from None


def mixer_class(kind: str) -> type:
    return _lookup(MIXERS, "mixer", kind)


def feed_forward_class(kind: str) -> type:
    return _lookup(FEED_FORWARDS, "feed-forward", kind)


def norm_class(kind: str) -> type:
    return _lookup(NORMS, "norm", kind)


def position_encoding_class(kind: str) -> type:
    return _lookup(POSITION_ENCODINGS, "position encoding", kind)


def block_class(kind: str) -> type:
    return _lookup(BLOCKS, "block", kind)


def embedding_class(kind: str) -> type:
    return _lookup(EMBEDDINGS, "embedding", kind)


def head_class(kind: str) -> type:
    return _lookup(HEADS, "head", kind)


def stream_op_class(kind: str) -> type:
    return _lookup(STREAM_OPS, "stream op", kind)
