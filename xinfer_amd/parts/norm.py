"""RMSNorm on the float32 residual stream, fused with the residual add.

out = s * rsqrt(mean(s^2) + eps) * w with s = resid (+ add), everything in float32 and
one rounding to the output type (reference: NormX::forward and forward_add,
/root/reference/src/models/layers/others.rs:22-62; weight kept in float32,
/root/reference/src/models/qwen3.rs:83).  With `weight_offset` c the stored tensor lies around -c + 1
and the factor is c + w (c = 1: the tensor is the factor's distance from one); the sum is made once, in float32, when the
tensor is loaded.  With `groups` G the row falls into G equal parts, each divided by its own root mean square; the weight is
as long as the row.  The pass over an open stream makes such a norm beside its sums (`parts/joining.py`); in other places it
takes a pass of its own.
"""
from __future__ import annotations

from typing import List, Optional

import torch

from .. import kernels
from ..config.spec import PartSpec
from ..weights.store import TensorDecl, WeightStore
from .base import Norm, register_norm


@register_norm("rmsnorm")
class RMSNorm(Norm):
    graph_safe = True
    joinable = True

    @property
    def foldable(self) -> bool:      # the products around it can carry it (parts.base.Folded)
        return self.groups == 1

    def __init__(self, spec: PartSpec, dtype: torch.dtype):
        super().__init__(spec, dtype)
        self.dim = int(spec["dim"])
        self.eps = float(spec["eps"])
        self.weight_offset = float(spec.get("weight_offset") or 0.0)
        self.groups = int(spec.get("groups") or 1)
        if self.groups < 1 or self.dim % self.groups:
            raise ValueError(f"a norm over {self.dim} in {self.groups} groups")
        self.weight: Optional[torch.Tensor] = None

    @classmethod
    def declare(cls, spec: PartSpec, prefix: str) -> List[TensorDecl]:
        # random weights lie around 1 - offset, so that the factor lies around 1 either way
        init = "norm" if not spec.get("weight_offset") else f"normal({1.0 - float(spec['weight_offset'])},0.1)"
        return [TensorDecl(f"{prefix}.weight" if "name" not in spec.params else spec["name"],
                           (int(spec["dim"]),), init)]

    def load(self, store: WeightStore, prefix: str, device) -> None:
        name = self.spec.get("name") or f"{prefix}.weight"
        w = store.get(name, torch.float32, device)
        self.weight = (w + self.weight_offset if self.weight_offset else w).contiguous()

    def forward(self, resid, add, out_dtype, rows=None, out=None, add_scale: float = 1.0):
        if self.groups > 1:
            terms = [] if add is None else [(add, None, 0.0, add_scale)]
            s, _, _, (h,) = kernels.stream_join(resid, terms, [(self.weight, self.eps, self.groups)], out_dtype,
                                                keep=bool(terms) and rows is None, rows=rows)
            if s is not None:
                resid.copy_(s)
            return h if out is None else out.copy_(h)
        return kernels.add_rmsnorm(resid, add, self.weight, self.eps, out_dtype, rows=rows, out=out, y_scale=add_scale)

    def forward_branch(self, resid, y, rows_dtype):
        if self.groups > 1:
            s, low, _, _ = kernels.stream_join(resid, [(y, self.weight, self.eps, 1.0, self.groups)], (), rows_dtype or torch.float32,
                                               keep=True, rounded=rows_dtype is not None)
            resid.copy_(s)
            return low
        return kernels.rmsnorm_add(resid, y, self.weight, self.eps, rows_dtype)
