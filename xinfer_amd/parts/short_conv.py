"""A short causal convolution per channel, with the last inputs of a request as state, and a mixer behind one.

`short_conv` runs it for a part: out[t] = act(bias + sum_j w[:, j] u[t - taps + 1 + j]), zeros before a sequence's start; a
request's slot of `tails` holds its last taps - 1 inputs (float32, oldest first) and is moved on by the step's tokens, in the
same launch where every sequence brings one token.

"input_conv" is a mixer that puts such a convolution in front of another mixer: what that one reads in place of h is

    h_t + sum_j w[:, j] h_(t - taps + 1 + j)          w [hidden, taps], no bias, no activation

The residual rides on the last tap: its weight is one larger (added once in float32, at load).  The last taps - 1 inputs h are
state of the request ("input_tail"), beside whatever the inner mixer keeps.  Parameters: hidden_size, taps, name (of the
tensor w), inner (the mixer's `PartSpec`).
"""
from __future__ import annotations

from typing import List, Optional, Tuple

import torch

from .. import kernels
from ..config.spec import PartSpec
from ..weights.store import TensorDecl, WeightStore
from .base import KVNeed, LayerCache, Mixer, StateNeed, StepContext, mixer_class, register_mixer, state_needs_of


def short_conv(u: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor, tails: Optional[torch.Tensor], ctx: StepContext,
               act: str = "silu", in_bias: Optional[torch.Tensor] = None, write: bool = True) -> torch.Tensor:
    """`tails` None: one tap, nothing is kept.  `write` False: the tails are read and stay as they are."""
    if tails is None:
        tails = torch.empty((1, 0, u.shape[1]), dtype=torch.float32, device=u.device)
        return kernels.causal_conv(u, weight, bias, tails, ctx.state_slots, ctx.tok_seq, ctx.cu_q, in_bias=in_bias, act=act)
    if write and ctx.max_q_len == 1 and ctx.num_tokens == ctx.num_seqs:
        return kernels.conv_step(u, weight, bias, tails, ctx.state_slots, in_bias=in_bias, act=act)
    out = kernels.causal_conv(u, weight, bias, tails, ctx.state_slots, ctx.tok_seq, ctx.cu_q, in_bias=in_bias, act=act)
    if write:
        kernels.conv_tail(u, tails, ctx.state_slots, ctx.cu_q, in_bias=in_bias)
    return out


@register_mixer("input_conv")
class InputConv(Mixer):
    TAIL = "input_tail"

    def __init__(self, spec: PartSpec, dtype: torch.dtype):
        super().__init__(spec, dtype)
        self.hidden = int(spec["hidden_size"])
        self.taps = int(spec["taps"])
        if min(self.hidden, self.taps) <= 0:
            raise ValueError(f"a convolution of {self.taps} taps over {self.hidden} channels cannot be run")
        inner = spec["inner"]
        self.inner: Mixer = mixer_class(inner.kind)(inner, dtype)
        self.weight: Optional[torch.Tensor] = None
        self.bias: Optional[torch.Tensor] = None

    @property
    def graph_safe(self) -> bool:
        return self.inner.graph_safe

    @classmethod
    def declare(cls, spec: PartSpec, prefix: str) -> List[TensorDecl]:
        inner = spec["inner"]
        return mixer_class(inner.kind).declare(inner, prefix) + [
            TensorDecl(spec["name"], (int(spec["hidden_size"]), int(spec["taps"])), "normal(0,0.3)")]

    def load(self, store: WeightStore, prefix: str, device) -> None:
        self.inner.load(store, prefix, device)
        w = store.get(self.spec["name"], torch.float32, device).clone()
        w[:, -1] += 1.0
        self.weight = w.contiguous()
        self.bias = torch.zeros(self.hidden, dtype=torch.float32, device=device)

    def cache_need(self) -> Optional[KVNeed]:
        return self.inner.cache_need()

    def state_need(self) -> Tuple[StateNeed, ...]:
        needs = state_needs_of(self.inner.state_need())       # the inner mixer's first: its own `LayerCache.state`
        if self.taps > 1:
            needs += (StateNeed((self.taps - 1, self.hidden), torch.float32, self.TAIL),)
        return needs or None

    def forward(self, x: torch.Tensor, ctx: StepContext, cache: LayerCache) -> torch.Tensor:
        tails = None
        if self.taps > 1:
            tails = cache.states.get(self.TAIL)
            if tails is None:
                raise RuntimeError("a convolution in front of a mixer was given no state slots")
        h = short_conv(x, self.weight, self.bias, tails, ctx, act="none", write=cache.write)
        return self.inner.forward(h, ctx, cache)
