"""A plain, slow Tisosun written from the design's equations: one function a mechanism, every token of a sequence at
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
def rms_norm(x, eps, w=None):
    """x / sqrt(mean(x^2) + eps) over the last axis, times w if given."""
    y = x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)
    return y if w is None else y * w


def layer_norm_weight(w):
    """A model norm's tensor holds its factor's distance from one: the factor is 1 + w."""
    return 1.0 + w


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


# ---- rotary positions: pairs (2i, 2i + 1), frequencies blended along a ramp ------------------------------
def rotary_frequencies(rot):
    """The frequencies of the pairs and the factor on cos and sin.  Without `scaling`: base^(-2i / dims) and 1."""
    d, base = rot["dims"], rot["base"]
    f = [base ** (-2.0 * i / d) for i in range(d // 2)]
    sc = rot.get("scaling")
    if not sc:
        return torch.tensor(f, dtype=torch.float64), 1.0

    def dim_of(turns):
        return d * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(dim_of(sc["fast"])), 0)
    hi = min(math.ceil(dim_of(sc["slow"])), d - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * r + fi * (1.0 - r))
    return torch.tensor(out, dtype=torch.float64), 0.1 * math.log(sc["factor"]) + 1.0


def rotate_pairs(x, rot, positions):
    """x [T, heads, n]: dims 2i and 2i + 1 of every head turn by p f_i; dims from rot.dims on pass unchanged."""
    f, grow = rotary_frequencies(rot)
    ang = positions.to(torch.float64)[:, None] * f[None, :]
    c, s = (ang.cos() * grow)[:, None, :].to(x.dtype), (ang.sin() * grow)[:, None, :].to(x.dtype)
    out = x.clone()
    d = rot["dims"]
    u, v = x[..., 0:d:2], x[..., 1:d:2]
    out[..., 0:d:2] = u * c - v * s
    out[..., 1:d:2] = v * c + u * s
    return out


# ---- attention within chunks ------------------------------------------------------------------------------
def chunk_seen(T, size):
    """[T, T]: query i sees key j if j <= i and both lie in the same chunk of `size` positions (None: every j <= i)."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    return seen if not size else seen & (i // size == j // size)


def capped(s, cap):
    return cap * torch.tanh(s / cap) if cap else s


def softmax_heads(q, k, v, scale, cap, size):
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H * dv]."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    seen = chunk_seen(T, size)
    out = []
    for h in range(H):
        g = h // (H // G)
        s = capped((q[:, h] @ k[:, g].T) * scale, cap).masked_fill(~seen, float("-inf"))
        out.append(torch.softmax(s, dim=-1) @ v[:, g])
    return torch.cat(out, dim=-1)


def attention_branch(h, w, m, eps, positions):
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = (h @ w["q"].T + w["q.b"]).view(T, H, d)
    k = (h @ w["k"].T + w["k.b"]).view(T, G, d)
    v = (h @ w["v"].T + w["v.b"]).view(T, G, dv)
    q, k = rms_norm(q, eps, w["q.norm"]), rms_norm(k, eps, w["k.norm"])
    if m.get("rot"):
        q, k = rotate_pairs(q, m["rot"], positions), rotate_pairs(k, m["rot"], positions)
    return softmax_heads(q, k, v, m["scale"], m.get("softcap"), (m.get("mask") or {}).get("size")) @ w["o"].T


# ---- linear attention with one constant decay a head ---------------------------------------------------------
def decayed_state(q, k, v, decay, S=None):
    """q, k [T, H, dk], v [T, H, dv]: S <- decay_h S + k v^T, o = S^T q.  Returns (o [T, H, dv], S)."""
    T, H, dk = q.shape
    S = torch.zeros(H, dk, v.shape[2], dtype=q.dtype) if S is None else S.clone()
    a = torch.tensor(decay, dtype=q.dtype)[:, None, None]
    o = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for t in range(T):
        S = a * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    return o, S


def lightning_branch(h, w, m, eps):
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q, k, v = silu(h @ w["q"].T).view(T, H, dk), silu(h @ w["k"].T).view(T, H, dk), silu(h @ w["v"].T).view(T, H, dv)
    o, _ = decayed_state(q, k, v, m["decay"])
    o = rms_norm(o.reshape(T, H * dv), eps, w["norm"])               # one mean over all heads
    return (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def sub(w, prefix):
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def parallel(h, w, m, eps, positions):
    left = attention_branch(h, sub(w, "left."), m["left"], eps, positions)
    right = lightning_branch(h, sub(w, "right."), m["right"], eps)
    return 0.5 * (rms_norm(left, eps, w["left.out"]) + rms_norm(right, eps, w["right.out"]))


# ---- gated recurrences, channel by channel -----------------------------------------------------------------
def channel_recurrence(a, b, S=None):
    """S_t = a_t S_(t-1) + b_t; a, b [T, C].  Returns (S_t for every t, the last one)."""
    S = torch.zeros(a.shape[1], dtype=a.dtype) if S is None else S.clone()
    out = torch.zeros_like(a)
    for t in range(a.shape[0]):
        S = a[t] * S + b[t]
        out[t] = S
    return out, S


def mingru_terms(z, u):
    """(a, b) from the gate's logit and the candidate's: a = 1 - sigmoid(z), b = sigmoid(z) * candidate."""
    g = torch.sigmoid(z)
    cand = torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    return 1.0 - g, g * cand


def mingru(h, w):
    a, b = mingru_terms(h @ w["z"].T + w["z.b"], h @ w["x"].T + w["x.b"])
    S, _ = channel_recurrence(a, b)
    return (S * silu(h @ w["g"].T)) @ w["o"].T


def short_conv(u, taps_w, bias):
    """u [T, C]; taps_w [C, taps]: y_t = bias + sum_j taps_w[:, j] u_(t - taps + 1 + j), nothing before a sequence."""
    T, C = u.shape
    taps = taps_w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, C, dtype=u.dtype), u], dim=0)
    out = bias[None, :].expand(T, C).clone()
    for j in range(taps):
        out = out + padded[j:j + T] * taps_w[:, j][None, :]
    return out


def block_gate(u, w, b):
    """u [T, C] in equal parts, w [blocks, C / blocks, C / blocks] ([out, in]), b [blocks, C / blocks] -> logits [T, C]."""
    n, s, _ = w.shape
    parts = [u[:, i * s:(i + 1) * s] @ w[i].T + b[i] for i in range(n)]
    return torch.cat(parts, dim=-1)


def rglru_terms(u, r_logit, i_logit, lam):
    """log a = -8 sigmoid(r) softplus(lam); (a, b) with b = sqrt(1 - a^2) * sigmoid(i) * u."""
    log_a = -8.0 * torch.sigmoid(r_logit) * softplus(lam)
    return torch.exp(log_a), torch.sqrt(-torch.expm1(2.0 * log_a)) * torch.sigmoid(i_logit) * u


def rglru(h, w):
    y = gelu_tanh(h @ w["y"].T + w["y.b"])
    u = short_conv(h @ w["x"].T + w["x.b"], w["conv"], w["conv.b"])
    a, b = rglru_terms(u, block_gate(u, w["ra"], w["ra.b"]), block_gate(u, w["ri"], w["ri.b"]), w["lam"])
    S, _ = channel_recurrence(a, b)
    return (S * y) @ w["o"].T


# ---- around the mixers ----------------------------------------------------------------------------------------
def dense_mlp(h, w):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def token_side(x, part, w, eps):
    """What a layer adds for the token itself: part [T, dim] is the layer's part of the token's row."""
    y = (gelu_tanh(x @ w["gate"].T) * part) @ w["proj"].T
    return rms_norm(y, eps, w["norm"])


def depth_average(weights, results):
    """sum_j weights[j] results[j]: results = [the embedding output, the layers' results so far]."""
    out = torch.zeros_like(results[0])
    for c, r in zip(weights, results):
        out = out + c * r
    return out


# ---- the model ---------------------------------------------------------------------------------------------
class PlainTisosun:
    def __init__(self, model_dir, dtype=torch.float64):
        with open(os.path.join(model_dir, "config.json")) as f:
            self.cfg = json.load(f)
        self.dtype = dtype
        self.w = {}
        with safe_open(os.path.join(model_dir, "model.safetensors"), "pt") as f:
            for name in f.keys():
                t = f.get_tensor(name)
                self.w[name] = t.to(dtype) if t.is_floating_point() else t

    def mixer(self, i, h, positions):
        l, eps = self.cfg["layers"][i], self.cfg["norm"]["eps"]
        w = sub(self.w, f"l{i}.mix.")
        if l["type"] == "parallel":
            return parallel(h, w, l["mixer"], eps, positions)
        if l["type"] == "rglru":
            return rglru(h, w)
        if l["type"] == "mingru":
            return mingru(h, w)
        raise ValueError(l["type"])

    def stream(self, tokens, averaged=True):
        """The embedding output, then for every layer what it hands on (`averaged`) or its own result."""
        cfg, eps = self.cfg, self.cfg["norm"]["eps"]
        tok = torch.tensor(tokens)
        positions = torch.arange(len(tokens))
        x = rms_norm(self.w["embed"][tok], eps, layer_norm_weight(self.w["embed.norm"]))
        results, out = [x], [x]
        dim = (cfg.get("token_side") or {}).get("dim")
        for i, l in enumerate(cfg["layers"]):
            branches = self.mixer(i, rms_norm(x, eps, layer_norm_weight(self.w[f"l{i}.norm1"])), positions)
            if l.get("mlp") is not None:
                h2 = rms_norm(x, eps, layer_norm_weight(self.w[f"l{i}.norm2"]))
                branches = branches + dense_mlp(h2, sub(self.w, f"l{i}.mlp."))
            x = x + branches
            if dim:
                part = self.w["side.embed"][tok][:, i * dim:(i + 1) * dim]
                x = x + token_side(x, part, sub(self.w, f"l{i}.side."), eps)
            results.append(x)
            x = depth_average(self.w[f"l{i}.dwa"], results)
            out.append(x if averaged else results[-1])
        return out

    def logits(self, tokens):
        x = self.stream(tokens)[-1]
        return rms_norm(x, self.cfg["norm"]["eps"], layer_norm_weight(self.w["final.norm"])) @ self.w["head"].T

    def greedy(self, prompt, n):
        ids = list(prompt)
        for _ in range(n):
            ids.append(int(self.logits(ids)[-1].argmax()))
        return ids[len(prompt):]
