"""Gated recurrences of one float32 number a channel, as mixers: "mingru" and "rglru".

Both keep, per request, a float32 vector S [width] in the request's state slot and do, token by token and channel by
channel, S_t = a_t S_(t-1) + b_t (`kernels.channel_scan`: single tokens and short portions in one walk, long portions in
chunks side by side), multiply S_t by a gate made of the token and project it (`o`).  A slot holds zeros when a request runs
its first token, and a step leaves the state after its last token there, so a prompt may be cut anywhere.

  mingru   a gated recurrence whose gates read only the current token: z = sigmoid(W_z h + b_z), u = W_x h + b_x, a = 1 - z,
           b = z * (u + 1/2 where u >= 0, sigmoid(u) where u < 0); the gate is silu(W_g h).
           Tensors: z, z.b, x, x.b, g, o.
  rglru    the recurrent block of Griffin: u = conv(W_x h + b_x), a causal convolution per channel over the last `conv`
           tokens with a bias and no activation; in each of `blocks` equal parts of u, r = sigmoid(R u + b_r) and i =
           sigmoid(I u + b_i) with square matrices R, I of the part; log a = -RATE r softplus(lam), a = exp(log a), b =
           sqrt(1 - a^2) i u, from S = 0 at the first token too; the gate is gelu_tanh(W_y h + b_y).  The convolution's
           last conv - 1 inputs are a second state of the request ("conv_tail", float32, oldest first).
           Tensors: y, y.b, x, x.b, conv [width, taps] (the last column is the current token's), conv.b, ra, ra.b, ri, ri.b
           ([blocks, part, part] as [out, in] and [blocks, part]), lam, o.

Gates, logarithms, exponentials, a, b and S are float32 in both precisions (the gates' products leave the matrix cores
as float32 sums); projections and the convolution's result are in the activation dtype.  The spec's `names` replaces any
tensor's name.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Tuple

import torch

from .. import kernels
from ..config.spec import PartSpec
from ..weights.store import TensorDecl, WeightStore
from .base import LayerCache, Mixer, StateNeed, StepContext, register_mixer
from .linear import Linear
from .short_conv import short_conv


class _ChannelState(Mixer):
    graph_safe = True
    NAMES: Dict[str, str] = {}

    def __init__(self, spec: PartSpec, dtype: torch.dtype):
        super().__init__(spec, dtype)
        self.hidden = int(spec["hidden_size"])
        self.width = int(spec["width"])
        if min(self.hidden, self.width) <= 0:
            raise ValueError(f"a recurrence of {self.width} channels on a width of {self.hidden} cannot be run")
        self.proj: Optional[Linear] = None
        self.o: Optional[Linear] = None

    @classmethod
    def _names(cls, spec: PartSpec, prefix: str) -> Dict[str, str]:
        given = spec.get("names") or {}
        return {k: f"{prefix}.{given.get(k, v)}" for k, v in cls.NAMES.items()}

    def _load_products(self, store: WeightStore, n: Dict[str, str], parts, device) -> None:
        lin = lambda k: store.get(n[k], None, device).to(self.dtype)
        self.proj = Linear(torch.cat([lin(k) for k in parts], dim=0))
        self.o = Linear(lin("o"))

    @staticmethod
    def _cutting(ctx: StepContext):
        """The portions' lengths where the host may read them (a step of single tokens reads nothing: it may be recorded)."""
        if ctx.max_q_len <= 1 or not ctx.cu_q_host:
            return {}
        cu = ctx.cu_q_host
        return dict(q_lens=[cu[b + 1] - cu[b] for b in range(ctx.num_seqs)], plan_cache=ctx.scratch)


@register_mixer("mingru")
class MinGRU(_ChannelState):
    NAMES = {"z": "z", "z_bias": "z.b", "x": "x", "x_bias": "x.b", "g": "g", "o": "o"}

    def __init__(self, spec: PartSpec, dtype: torch.dtype):
        super().__init__(spec, dtype)
        self.z_bias = self.x_bias = None

    @classmethod
    def declare(cls, spec: PartSpec, prefix: str) -> List[TensorDecl]:
        h, w = int(spec["hidden_size"]), int(spec["width"])
        n = cls._names(spec, prefix)
        return [TensorDecl(n["z"], (w, h)), TensorDecl(n["z_bias"], (w,), "normal(-1,1)"), TensorDecl(n["x"], (w, h)),
                TensorDecl(n["x_bias"], (w,), "normal(0,0.1)"), TensorDecl(n["g"], (w, h)), TensorDecl(n["o"], (h, w))]

    def load(self, store: WeightStore, prefix: str, device) -> None:
        n = self._names(self.spec, prefix)
        self._load_products(store, n, ("z", "x", "g"), device)
        self.z_bias = store.get(n["z_bias"], torch.float32, device).contiguous()
        self.x_bias = store.get(n["x_bias"], torch.float32, device).contiguous()

    def state_need(self) -> StateNeed:
        return StateNeed((self.width,), torch.float32)

    def forward(self, x: torch.Tensor, ctx: StepContext, cache: LayerCache) -> torch.Tensor:
        if cache.state is None:
            raise RuntimeError("a gated recurrence was given no state slots")
        w = self.width
        p = self.proj(x, out_dtype=self.dtype)
        y = kernels.channel_scan(p[:, 2 * w:], "silu", cache.state, ctx.state_slots, ctx.cu_q,
                                 mingru=(p[:, :w], self.z_bias, p[:, w:2 * w], self.x_bias), **self._cutting(ctx))
        return self.o(y, out_dtype=self.dtype, allow_split=True)


@register_mixer("rglru")
class RealGatedRecurrence(_ChannelState):
    RATE = 8.0                # the largest decay's exponent, times softplus(lam)
    NAMES = {"y": "y", "y_bias": "y.b", "x": "x", "x_bias": "x.b", "conv": "conv", "conv_bias": "conv.b", "r": "ra", "r_bias": "ra.b",
             "i": "ri", "i_bias": "ri.b", "lam": "lam", "o": "o"}

    def __init__(self, spec: PartSpec, dtype: torch.dtype):
        super().__init__(spec, dtype)
        self.taps = int(spec["conv"])
        self.blocks = int(spec["blocks"])
        if self.taps <= 0 or self.blocks <= 0 or self.width % self.blocks:
            raise ValueError(f"{self.width} channels in {self.blocks} blocks behind {self.taps} taps cannot be run")
        self.gates: Optional[torch.Tensor] = None         # [blocks, 2, part, part]: the r gate's matrix, then the i gate's
        self.y_bias = self.x_bias = self.conv_w = self.conv_b = self.r_bias = self.i_bias = self.rate = None

    @classmethod
    def declare(cls, spec: PartSpec, prefix: str) -> List[TensorDecl]:
        h, w, taps, k = (int(spec[v]) for v in ("hidden_size", "width", "conv", "blocks"))
        part = w // k
        n = cls._names(spec, prefix)
        return [TensorDecl(n["y"], (w, h)), TensorDecl(n["y_bias"], (w,), "normal(0,0.1)"), TensorDecl(n["x"], (w, h)),
                TensorDecl(n["x_bias"], (w,), "normal(0,0.1)"), TensorDecl(n["conv"], (w, taps), "normal(0,0.5)"),
                TensorDecl(n["conv_bias"], (w,), "normal(0,0.1)"), TensorDecl(n["r"], (k, part, part)),
                TensorDecl(n["r_bias"], (k, part), "normal(0,0.5)"), TensorDecl(n["i"], (k, part, part)),
                TensorDecl(n["i_bias"], (k, part), "normal(0,0.5)"), TensorDecl(n["lam"], (w,), "normal(-4,1)"),
                TensorDecl(n["o"], (h, w))]

    def load(self, store: WeightStore, prefix: str, device) -> None:
        n = self._names(self.spec, prefix)
        self._load_products(store, n, ("y", "x"), device)
        f32 = lambda k: store.get(n[k], torch.float32, device).reshape(-1).contiguous()
        self.y_bias, self.x_bias, self.conv_b, self.r_bias, self.i_bias = (f32(k) for k in ("y_bias", "x_bias", "conv_bias", "r_bias", "i_bias"))
        self.conv_w = store.get(n["conv"], torch.float32, device).contiguous()
        self.gates = torch.stack([store.get(n[k], None, device).to(self.dtype) for k in ("r", "i")], dim=1).contiguous()
        lam = store.get(n["lam"], torch.float32, device).double()
        softplus = torch.clamp(lam, min=0.0) + torch.log1p(torch.exp(-lam.abs()))
        self.rate = (-self.RATE * softplus).float().contiguous()

    def state_need(self) -> Tuple[StateNeed, ...]:
        needs = [StateNeed((self.width,), torch.float32, "state")]
        if self.taps > 1:
            needs.append(StateNeed((self.taps - 1, self.width), torch.float32, "conv_tail"))
        return tuple(needs)

    def forward(self, x: torch.Tensor, ctx: StepContext, cache: LayerCache) -> torch.Tensor:
        if cache.state is None or (self.taps > 1 and "conv_tail" not in cache.states):
            raise RuntimeError("a gated recurrence was given no state slots")
        w = self.width
        p = self.proj(x, out_dtype=self.dtype)
        u = short_conv(p[:, w:], self.conv_w, self.conv_b, cache.states["conv_tail"] if self.taps > 1 else None, ctx,
                       in_bias=self.x_bias, act="none")
        terms = kernels.rglru_terms(u, self.gates, self.r_bias, self.i_bias, self.rate)
        y = kernels.channel_scan(p[:, :w], "gelu_tanh", cache.state, ctx.state_slots, ctx.cu_q, ready=terms, gate_bias=self.y_bias,
                                 **self._cutting(ctx))
        return self.o(y, out_dtype=self.dtype, allow_split=True)
