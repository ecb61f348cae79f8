"""An open stream brought up to date: its branch outputs and terms added, the average over the depth taken, and the norms
that follow made, in one pass over the rows (`kernels.stream_join`)."""
from __future__ import annotations

from dataclasses import replace
from typing import List, Optional, Sequence, Tuple

import torch

from .. import kernels
from .base import Norm, Stream, Term


def joins(*norms: Norm) -> bool:
    """Whether the pass can make these norms itself: their form is x / sqrt(mean(x^2) + eps) * weight, over the row or over
    equal parts of it."""
    return len(norms) <= kernels.JOIN_NORMS and all(n.foldable or n.joinable for n in norms)


def join(stream: Stream, dtype: torch.dtype, norms: Sequence[Norm] = (), rounded: bool = False,
         rows: Optional[torch.Tensor] = None) -> Tuple[Stream, Optional[torch.Tensor], List[torch.Tensor]]:
    """Returns (the stream with nothing left to add, its rows in `dtype` if `rounded`, the rows normed by each of `norms`
    in `dtype`).  The stream's tensor is not changed: the new one is another.  `rows` (int32): only these rows are made, and
    only their norms; the stream that comes back is then the one that was given."""
    if stream.folded is not None:
        raise RuntimeError("the stream carries a half-done norm of the block before")
    terms = () if stream.pending is None else (Term(stream.pending, scale=stream.pending_scale),)
    terms = [(t.y, t.weight, t.eps, t.scale, t.groups) for t in terms + tuple(stream.terms)]
    weighed = [(n.weight, n.eps, getattr(n, "groups", 1)) for n in norms]
    x = stream.resid
    while (sum(t[1] is None for t in terms) > kernels.JOIN_PLAIN or sum(t[1] is not None for t in terms) > kernels.JOIN_NORMED):
        first = next(t for t in terms if (t[1] is None) == (sum(u[1] is None for u in terms) > kernels.JOIN_PLAIN))
        x = kernels.stream_join(x, [first], keep=True)[0]          # more terms than one launch takes: one ahead
        terms.remove(first)
    avg, result = stream.average, None
    if avg is not None:
        result = avg.results[avg.place]
    if rows is not None:
        _, _, _, outs = kernels.stream_join(x, terms, weighed, dtype, rows=rows,
                                            average=None if avg is None else (avg.first, avg.results, avg.place, avg.weights))
        return stream, None, outs
    if not terms and avg is None:                # nothing to add
        low = x
        if rounded and dtype != torch.float32:
            low = kernels.stream_join(x, out_dtype=dtype, rounded=True)[1]
        outs = kernels.stream_join(x, [], weighed, dtype)[3] if weighed else []
        return Stream(x), (low if rounded else None), outs
    same = rounded and dtype == torch.float32    # float32: the stream is its own rows
    s, low, u, outs = kernels.stream_join(
        x, terms, weighed, dtype, keep=True, result=result, rounded=rounded and not same and avg is None,
        average=None if avg is None else (avg.first, avg.results, avg.place, avg.weights))
    new = s if avg is None else u
    if rounded and avg is not None and not same:
        low = kernels.stream_join(new, out_dtype=dtype, rounded=True)[1]
    return Stream(new), (new if same else low), outs


def closed(stream: Stream) -> Stream:
    """The stream for a part that knows nothing of open ones."""
    if not stream.open:
        return stream
    return join(replace(stream, rows=None), torch.float32)[0]
