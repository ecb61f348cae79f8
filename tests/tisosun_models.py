"""Small Tisosun configurations for tests, and the maker of their model folders.

A: every mixer type in the order rglru, parallel, mingru, parallel; 3 query heads a kv head; values wider than keys; half of
   a head turned, with blended frequencies; chunks of 21 positions on pages of 16; a layer without feed-forward; 3 taps.
B: the values another model may make equal or 1: as many kv heads as heads, values as long as keys, whole heads turned
   without scaling, chunks as long as a page, no soft cap, one head of the linear attention, one block of gates, one tap,
   recurrences as wide as the model.  (A token input of one column is tested alone: its norm
   leaves a sign, which no rounding keeps near zero.)
C: sizes in no kernel's favourite multiples (width 50, heads of 12 and 20, recurrences of 33 and 42 channels in blocks of 6),
   one kv head, chunks of 5 (shorter than a page) and of 1, 6 taps, no token input, no rotation in one layer.
M: recurrences alone (no layer keeps pages): requests have states and lengths, and no cache to read.
R: real-looking head sizes with pages of 64, for the matrix-core kernels: keys of 64 with values of 48, keys and values of 128
   (the vectorized kernel for the heads), gates in blocks of 128, chunks of 100 and 150.
S: the matrix-core kernels' sizes again: one kv head of 64 under eight heads (single tokens take the heads as the rows of
   a block), chunks of 70, a layer whose chunks are wider than any request, a layer that sees every token, a block of 72
   channels (three tiles of gates, the last in part), a feed-forward in no layer but one.
"""
import os

import torch


def _rot(dims, base, scaling=None):
    out = {"dims": dims, "base": base}
    if scaling:
        out["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return out


def _left(heads, kv_heads, dim, vdim, scale, chunk=None, cap=None, rot=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if cap:
        m["softcap"] = cap
    if chunk:
        m["mask"] = {"size": chunk}
    if rot:
        m["rot"] = rot
    return m


def _right(dim, vdim, decay):
    return {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}


def _mlp(ff):
    return None if ff is None else {"kind": "dense", "ff": ff}


def _par(left, right, ff):
    return {"type": "parallel", "mixer": {"left": left, "right": right}, "mlp": _mlp(ff)}


def _rg(width, blocks, conv, ff):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": conv}, "mlp": _mlp(ff)}


def _mg(width, ff):
    return {"type": "mingru", "mixer": {"width": width}, "mlp": _mlp(ff)}


def _config(vocab, width, eps, side, layers):
    out = {"architecture": "Tisosun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if side:
        out["token_side"] = {"dim": side}
    return out


MODELS = {
    "A": dict(config=_config(311, 96, 1e-5, 12, [
        _rg(120, 3, 3, 160),
        _par(_left(6, 2, 16, 24, 0.4, 21, 15.0, _rot(8, 500.0, (4.0, 64, 8.0, 1.0))), _right(12, 20, (0.6, 0.97, 0.9995)), 128),
        _mg(72, None),
        _par(_left(4, 2, 8, 16, 0.5, 34, 30.0, _rot(4, 100.0)), _right(8, 24, (0.9, 0.999)), 96)]),
        seed=41, linear_std=0.08, norm_std=0.1, page_size=16),
    "B": dict(config=_config(257, 100, 1e-6, 8, [
        _par(_left(5, 5, 20, 20, 0.35, 8, None, _rot(20, 10000.0)), _right(20, 20, (0.98,)), 72),
        _rg(100, 1, 1, 100),
        _mg(100, 60)]),
        seed=47, linear_std=0.1, norm_std=0.2, page_size=8),
    "C": dict(config=_config(131, 50, 1e-5, None, [
        _mg(33, 34),
        _par(_left(3, 1, 12, 20, 0.5, 5, 8.0, _rot(6, 50.0, (2.5, 30, 4.0, 0.5))), _right(6, 10, (0.5, 0.8, 0.95, 0.99, 1.0)), 40),
        _rg(42, 7, 6, None),
        _par(_left(2, 1, 10, 6, 0.6, 1, 20.0), _right(14, 6, (0.7, 0.996)), 22)]),
        seed=43, linear_std=0.12, norm_std=0.1, page_size=8),
    "M": dict(config=_config(190, 72, 1e-6, 6, [
        _rg(64, 4, 4, 48), _mg(96, 64), _rg(80, 2, 2, None), _mg(40, 32)]),
        seed=44, linear_std=0.1, norm_std=0.15, page_size=8),
    "R": dict(config=_config(409, 384, 1e-6, 32, [
        _par(_left(6, 2, 64, 48, 0.11, 100, 25.0, _rot(32, 20000.0, (3.0, 512, 16.0, 1.0))), _right(64, 96, (0.7, 0.995)), 512),
        _rg(512, 4, 4, 768),
        _par(_left(4, 2, 128, 128, 0.09, 150, 40.0, _rot(128, 50000.0)), _right(128, 64, (0.95, 0.9999)), 384),
        _mg(448, 256)]),
        seed=45, linear_std=0.04, norm_std=0.1, page_size=64),
    "S": dict(config=_config(300, 320, 1e-5, 16, [
        _par(_left(8, 1, 64, 64, 0.12, 70, None, _rot(48, 5000.0)), _right(32, 32, (0.8, 0.9, 0.99)), None),
        _par(_left(8, 1, 64, 96, 0.1, 1000, 12.0, _rot(64, 9000.0, (6.0, 200, 10.0, 2.0))), _right(16, 64, (0.99,)), 320),
        _rg(144, 2, 5, None),
        _par(_left(4, 4, 32, 32, 0.2, None, 9.0, _rot(16, 700.0)), _right(48, 40, (0.3, 0.998)), None)]),
        seed=46, linear_std=0.05, norm_std=0.1, page_size=64),
}


def make_model(model_dir, name):
    """Writes the folder of configuration `name`: random weights whose gates move with the token and whose recurrences reach
    far back; returns the folder."""
    from safetensors import safe_open
    from safetensors.torch import save_file
    from xinfer_amd.weights import write_random_model
    t = MODELS[name]
    write_random_model(model_dir, t["config"], t["seed"], t["linear_std"], t["norm_std"])
    path = os.path.join(model_dir, "model.safetensors")
    W = {}
    with safe_open(path, framework="pt") as f:
        for k in f.keys():
            W[k] = f.get_tensor(k).clone()
    for k in W:
        if k.endswith((".mix.ra", ".mix.ri", ".mix.z", ".side.gate", ".side.proj")):
            W[k] = (W[k].float() * 3).to(torch.bfloat16)
        if k.endswith(".side.norm"):             # a token's own input below the branches: its norm makes a small one large
            W[k] = (W[k].float() * 0.5).to(torch.bfloat16)
        if k.endswith(("left.q.b", "left.k.b", "left.v.b")):             # biases that matter beside the products
            W[k] = (W[k].float() * 6).to(torch.bfloat16)
    save_file({k: v.contiguous() for k, v in W.items()}, path)
    return model_dir
