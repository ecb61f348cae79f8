"""A plain, slow Litizen written from the design's equations: one function a mechanism, every token of a sequence at
once, no cache, no batching, no kernels.  It reads a model folder by itself (config.json, model.safetensors through the
safetensors library) and shares no code with the engine.

Notation: x the residual stream [T, width], h a sublayer's input, p a token's position (from 0).
"""
import json
import math
import os

import torch
from safetensors import safe_open


# ---- small functions ---------------------------------------------------------------------------------
def group_norm(x, eps, w=None, groups=1):
    """Each of `groups` equal parts of the last axis divided by its own sqrt(mean(part^2) + eps), times w over the whole."""
    p = x.reshape(*x.shape[:-1], groups, x.shape[-1] // groups)
    y = (p / torch.sqrt((p * p).mean(dim=-1, keepdim=True) + eps)).reshape(x.shape)
    return y if w is None else y * w


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def capped(s, cap):
    return cap * torch.tanh(s / cap) if cap else s


def causal_conv(u, taps_w):
    """u [T, C], taps_w [C, taps]: y_t = sum_j taps_w[:, j] u_(t - taps + 1 + j), nothing before a sequence's start."""
    T, C = u.shape
    taps = taps_w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, C, dtype=u.dtype), u], dim=0)
    out = torch.zeros_like(u)
    for j in range(taps):
        out = out + padded[j:j + T] * taps_w[:, j][None, :]
    return out


def input_conv(h, taps_w):
    """What a mixer reads in place of its input: the input plus its causal convolution."""
    return h + causal_conv(h, taps_w)


# ---- rotary positions, halves ---------------------------------------------------------------------------
def angles(base, dims, positions):
    """[T, dims / 2]: p * base^(-2i / dims)."""
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    return positions.to(torch.float64)[:, None] * f[None, :]


def turn_halves(x, ang):
    """x [T, heads, n]: dims i and i + half of every head turn by ang[t, i], half = ang.shape[1]; further dims pass."""
    half = ang.shape[1]
    c, s = ang.cos()[:, None, :].to(x.dtype), ang.sin()[:, None, :].to(x.dtype)
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], dim=-1)


# ---- which keys a query sees ------------------------------------------------------------------------------
def window_seen(T, size):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) if not size else (j <= i) & (i - j < size)


def chunk_seen(T, size):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) if not size else (j <= i) & (i // size == j // size)


def softmax_heads(q, k, v, scale, seen, sinks, cap=None):
    """q [T, H, d], k [T, G, d], v [T, G, dv], sinks [H] (each adds exp(sink) to its head's denominator) -> [T, H, dv]."""
    H, G = q.shape[1], k.shape[1]
    out = []
    for h in range(H):
        g = h // (H // G)
        s = capped((q[:, h] @ k[:, g].T) * scale, cap).masked_fill(~seen, float("-inf"))
        m = torch.maximum(s.max(dim=-1, keepdim=True).values, sinks[h])
        e = torch.exp(s - m)
        out.append((e / (e.sum(dim=-1, keepdim=True) + torch.exp(sinks[h] - m))) @ v[:, g])
    return torch.stack(out, dim=1)


# ---- mixers -------------------------------------------------------------------------------------------------
def attention(h, w, m, eps, positions):
    """Keys that are values too, a window, a sink of score 0."""
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    T = h.shape[0]
    q, k = (h @ w["q"].T).view(T, H, d), (h @ w["k"].T).view(T, G, d)
    v = k
    q, k = group_norm(q, eps, w["q.norm"]), group_norm(k, eps, w["k.norm"])
    if m.get("rot"):
        a = angles(m["rot"]["base"], m["rot"]["dims"], positions)
        q, k = turn_halves(q, a), turn_halves(k, a)
    o = softmax_heads(q, k, v, m["scale"], window_seen(T, (m.get("mask") or {}).get("size")), torch.zeros(H, dtype=h.dtype))
    return (o.reshape(T, H * d) * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def attention_turned(h, w, m, positions):
    """Values turned by their own position and turned back by the query's, chunks, a learned sink, a soft cap."""
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q, k, v = (h @ w["q"].T).view(T, H, d), (h @ w["k"].T).view(T, G, d), (h @ w["v"].T).view(T, G, dv)
    if m.get("rot"):
        a, av = angles(m["rot"]["base"], m["rot"]["dims"], positions), angles(m["rot"]["base"], dv, positions)
        q, k, v = turn_halves(q, a), turn_halves(k, a), turn_halves(v, av)
    o = softmax_heads(q, k, v, m["scale"], chunk_seen(T, (m.get("mask") or {}).get("size")), w["sink"], m.get("softcap"))
    if m.get("rot"):
        o = turn_halves(o, -av)
    return (o.reshape(T, H * dv) * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def state_walk(xs, B, C, d, a_log, skip, S=None):
    """xs [T, H, dv], B and C [T, H, N], d [T, H]: S <- exp(-exp(a_log) d) S + d B x^T, y = S^T C + skip x."""
    T, H, dv = xs.shape
    S = torch.zeros(H, B.shape[2], dv, dtype=xs.dtype) if S is None else S.clone()
    y = torch.zeros_like(xs)
    for t in range(T):
        S = torch.exp(-torch.exp(a_log) * d[t])[:, None, None] * S + d[t][:, None, None] * B[t][:, :, None] * xs[t][:, None, :]
        y[t] = (S * C[t][:, :, None]).sum(1) + skip[:, None] * xs[t]
    return y, S


def mamba2(h, w, m, eps):
    H, dv, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    T, inner = h.shape[0], H * dv
    p = h @ w["in"].T
    z, u, dt = p[:, :inner], p[:, inner:2 * inner + 2 * G * N], p[:, 2 * inner + 2 * G * N:]
    u = silu(causal_conv(u, w["conv"]) + w["conv.b"])
    x = u[:, :inner].view(T, H, dv)
    B = u[:, inner:inner + G * N].view(T, G, N).repeat_interleave(H // G, dim=1)
    C = u[:, inner + G * N:].view(T, G, N).repeat_interleave(H // G, dim=1)
    y, _ = state_walk(x, B, C, softplus(dt + w["dt_bias"]), w["A_log"], w["D"])
    return group_norm(y.reshape(T, inner) * silu(z), eps, w["norm"], m["norm_groups"]) @ w["o"].T


# ---- feed-forwards ----------------------------------------------------------------------------------------
def gated(h, w):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def route(h, router, correction, top):
    """(chosen [T, top], weights [T, top]): chosen by softmax scores + correction, weighted by the scores alone."""
    s = torch.softmax(h @ router.T, dim=-1)
    chosen = torch.topk(s + correction, top, dim=-1).indices
    wt = torch.gather(s, 1, chosen)
    return chosen, wt / (wt.sum(dim=-1, keepdim=True) + 1e-20)


def sub(w, prefix):
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def experts(h, w, mlp):
    n, idle = mlp["router"]["experts"], mlp["router"].get("identity", 0)
    chosen, wt = route(h, w["router"], w["correction"], mlp["router"]["top"])
    assert w["router"].shape[0] == n + idle
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, c in zip(chosen[t].tolist(), wt[t]):
            out[t] = out[t] + c * (h[t] if e >= n else gated(h[t], sub(w, f"e{e}.")))
    return out + gated(h, sub(w, "shared.")) if mlp.get("shared") else out


def feed_forward(h, w, mlp):
    return gated(h, w) if mlp["kind"] == "dense" else experts(h, w, mlp)


# ---- the model ---------------------------------------------------------------------------------------------
class PlainLitizen:
    def __init__(self, model_dir, dtype=torch.float64):
        with open(os.path.join(model_dir, "config.json")) as f:
            self.cfg = json.load(f)
        self.dtype = dtype
        self.w = {}
        with safe_open(os.path.join(model_dir, "model.safetensors"), "pt") as f:
            for name in f.keys():
                t = f.get_tensor(name)
                self.w[name] = t.to(dtype) if t.is_floating_point() else t

    def norm(self, x, name):
        return group_norm(x, self.cfg["norm"]["eps"], self.w[name], self.cfg["norm"].get("groups", 1))

    def mixer(self, i, h, positions):
        l, eps = self.cfg["layers"][i], self.cfg["norm"]["eps"]
        w = sub(self.w, f"l{i}.mix.")
        if l["type"] == "attention":
            return attention(h, w, l["mixer"], eps, positions)
        if l["type"] == "attention_2":
            return attention_turned(h, w, l["mixer"], positions)
        if l["type"] == "mamba2":
            return mamba2(h, w, l["mixer"], eps)
        raise ValueError(l["type"])

    def stream(self, tokens):
        """The embedding's output, then the stream after every layer."""
        cfg = self.cfg
        positions = torch.arange(len(tokens))
        x = self.w["embed"][torch.tensor(tokens)] * (cfg.get("embedding") or {}).get("scale", 1.0)
        out = [x]
        for i, l in enumerate(cfg["layers"]):
            h = input_conv(self.norm(x, f"l{i}.norm1"), self.w[f"l{i}.canon1"]) if cfg.get("canon") else self.norm(x, f"l{i}.norm1")
            x = x + self.norm(self.mixer(i, h, positions), f"l{i}.norm1b")
            if l.get("mlp") is not None:
                y = feed_forward(self.norm(x, f"l{i}.norm2"), sub(self.w, f"l{i}.mlp."), l["mlp"])
                x = x + self.norm(y, f"l{i}.norm2b")
            out.append(x)
        return out

    def logits(self, tokens):
        return capped(self.norm(self.stream(tokens)[-1], "final.norm") @ self.w["head"].T, self.cfg.get("logit_softcap"))

    def greedy(self, prompt, n):
        ids = list(prompt)
        for _ in range(n):
            ids.append(int(self.logits(ids)[-1].argmax()))
        return ids[len(prompt):]
