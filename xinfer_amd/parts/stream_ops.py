"""What may run on the residual stream between two runs of layers (`ScheduleEntry.before` and `after`).

"pass_start": what a pass over a span of layers adds to the stream when it starts,

    x <- x (+ the branch that is still to be added) (+ the embedding's output, `add_first`) + table[row]

with `table` a tensor [rows, dim] named by the spec and `row` the number of the pass.  One float32 kernel; the
stream goes on with nothing pending.

"token_side": a layer's own input for the token, behind its branches: with e the layer's part of a row of a table [vocab,
layers * dim] (`table`; columns `offset` .. `offset + dim`, row the token's id),

    x <- x + (y / sqrt(mean(y^2) + eps)) * norm,    y = W_proj (gelu_tanh(W_gate x) * e)

The products read x rounded to the activation dtype; x, the norm and the sum are float32.  Tensors `<prefix>.gate`, `.proj`,
`.norm` and the table, which the layers share.

"depth_average": what goes on is a weighted sum of the embedding's output and of all the layers' results so far, this one
included (tensor `name` [place + 2], place = how many results there were before it):

    x <- w[0] X_0 + w[1] X_1 + ... + w[place + 1] X_(place + 1)

The results of a step's layers are kept side by side in float32 for the length of the step; they are no state of a request.
Both leave their sums to whoever reads the stream next (`Stream.terms`, `Stream.average`).
"""
from __future__ import annotations

from dataclasses import replace
from typing import List, Optional

import torch

from .. import kernels
from ..config.spec import PartSpec
from ..weights.store import TensorDecl, WeightStore
from .base import DepthAverage, StepContext, Stream, StreamOp, Term, register_stream_op
from .joining import join
from .linear import Linear


@register_stream_op("pass_start")
class PassStart(StreamOp):
    graph_safe = True

    def __init__(self, spec: PartSpec, dtype: torch.dtype):
        super().__init__(spec, dtype)
        self.dim = int(spec["dim"])
        self.rows = int(spec.get("rows") or 0)          # 0: no table
        self.row = int(spec.get("row") or 0)
        self.needs_first = bool(spec.get("add_first", False))
        if self.rows and not (0 <= self.row < self.rows):
            raise ValueError(f"row {self.row} of a table of {self.rows}")
        self.vec: Optional[torch.Tensor] = None

    @classmethod
    def declare(cls, spec: PartSpec, prefix: str = "") -> List[TensorDecl]:
        if not int(spec.get("rows") or 0):
            return []
        return [TensorDecl(spec["name"], (int(spec["rows"]), int(spec["dim"])))]

    def load(self, store: WeightStore, prefix: str, device) -> None:
        if self.rows:
            self.vec = store.get(self.spec["name"], torch.float32, device)[self.row].contiguous()

    def forward(self, stream: Stream, first: Optional[torch.Tensor], ctx: StepContext) -> Stream:
        if stream.folded is not None:
            raise RuntimeError("the stream carries a half-done norm of the block before")
        if self.needs_first and first is None:
            raise RuntimeError("the embedding's output was not kept for the start of a pass")
        kernels.stream_start(stream.resid, stream.pending, stream.pending_scale, first if self.needs_first else None, self.vec)
        return Stream(stream.resid, None)


@register_stream_op("token_side")
class TokenSide(StreamOp):
    graph_safe = True
    writes_stream = False
    takes_open = True

    def __init__(self, spec: PartSpec, dtype: torch.dtype):
        super().__init__(spec, dtype)
        self.hidden = int(spec["hidden_size"])
        self.dim = int(spec["dim"])
        self.offset = int(spec["offset"])
        self.eps = float(spec["norm_eps"])
        if self.dim <= 0 or self.offset < 0 or self.offset + self.dim > int(spec["row"]):
            raise ValueError(f"columns {self.offset} .. {self.offset + self.dim} of a table row of {spec['row']}")
        self.gate: Optional[Linear] = None
        self.proj: Optional[Linear] = None
        self.norm_w = self.table = None

    @classmethod
    def declare(cls, spec: PartSpec, prefix: str = "") -> List[TensorDecl]:
        h, d, p = int(spec["hidden_size"]), int(spec["dim"]), spec["prefix"]
        return [TensorDecl(spec["table"], (int(spec["vocab_size"]), int(spec["row"])), "normal(0,1)"), TensorDecl(f"{p}.gate", (d, h)),
                TensorDecl(f"{p}.proj", (h, d)), TensorDecl(f"{p}.norm", (h,), "norm")]

    def load(self, store: WeightStore, prefix: str, device) -> None:
        p = self.spec["prefix"]
        self.table = store.shared(self.spec["table"], self.dtype, device)
        self.gate = Linear(store.get(f"{p}.gate", None, device).to(self.dtype))
        self.proj = Linear(store.get(f"{p}.proj", None, device).to(self.dtype))
        self.norm_w = store.get(f"{p}.norm", torch.float32, device).contiguous()

    def forward(self, stream: Stream, first: Optional[torch.Tensor], ctx: StepContext) -> Stream:
        stream, rows, _ = join(stream, self.dtype, rounded=True)
        if kernels.side_gate_takes(rows.shape[0], self.hidden, self.dtype):
            g = kernels.side_gate(rows, self.gate.weight, self.table, self.offset, ctx.ids)
        else:
            g = kernels.side_mul(self.gate(rows, out_dtype=self.dtype, allow_split=True), self.table, self.offset, ctx.ids)
        y = self.proj(g, out_dtype=self.dtype, allow_split=True)
        return replace(stream, terms=(Term(y, self.norm_w, self.eps),))


@register_stream_op("depth_average")
class DepthAveraging(StreamOp):
    graph_safe = True
    writes_stream = False
    takes_open = True
    needs_first = True

    def __init__(self, spec: PartSpec, dtype: torch.dtype):
        super().__init__(spec, dtype)
        self.place = int(spec["place"])           # results before this one
        self.layers = int(spec["layers"])         # results of a step
        if not (0 <= self.place < self.layers):
            raise ValueError(f"result {self.place} of {self.layers}")
        self.weights: Optional[torch.Tensor] = None

    @classmethod
    def declare(cls, spec: PartSpec, prefix: str = "") -> List[TensorDecl]:
        n = int(spec["place"]) + 2
        return [TensorDecl(spec["name"], (n,), f"normal({1.0 / n},0.05)")]

    def load(self, store: WeightStore, prefix: str, device) -> None:
        self.weights = store.get(self.spec["name"], torch.float32, device).contiguous()

    def forward(self, stream: Stream, first: Optional[torch.Tensor], ctx: StepContext) -> Stream:
        if first is None:
            raise RuntimeError("the embedding's output was not kept for the average over the depth")
        if stream.average is not None:
            stream = join(stream, self.dtype)[0]
        results = ctx.scratch.get("depth_results")
        if results is None or results.shape[0] != self.layers:
            results = torch.empty((self.layers, *first.shape), dtype=torch.float32, device=first.device)
            ctx.scratch["depth_results"] = results
        return replace(stream, rows=None, average=DepthAverage(first, results, self.place, self.weights))
