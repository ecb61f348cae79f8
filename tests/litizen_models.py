"""Small Litizen configurations for tests, and the maker of their model folders.

A: every mixer type, dense and routed feed-forwards and none; 3 query heads a kv head; values wider than keys; part of a head
   turned; chunks of 21 and windows of 19 positions on pages of 16; norms in 3 groups; 3 taps in front of the mixers, 4 in the
   state space; one identity expert.
B: the values another model may make equal or 1: as many kv heads as heads, whole heads turned, windows of 1, chunks as long as a
   page, one group of everything, one tap everywhere, one expert of three, no identity experts, no shared expert, no caps, an
   embedding without a factor.
C: sizes in no kernel's favourite multiples (width 50 in 5 groups of 10, heads of 12, 20 and 10, states of 7, experts of 22), one
   kv head, chunks of 5 (shorter than a page), windows of 3, 6 taps, all experts chosen.
M: state spaces alone (no layer keeps pages), with groups and norm groups as many as heads.
R: real-looking head sizes with pages of 64, for the matrix-core kernels: heads of 64 and 128, keys of 64 with values of 96, windows
   of 100, chunks of 150, norms in 4 groups of 96, eight experts with three identity experts.
S: the matrix-core kernels' sizes again: one kv head of 64 under eight heads (single tokens take the heads as the rows of a
   block) in both attentions, a window wider than any request, layers that see every token, no turning in one layer.

Random routers would leave some token's choice of experts to a difference that bfloat16 does not keep: `make_model` writes
weights in which a few columns of the stream (markers) are the embedding's alone (the norms behind the sublayers are zero
there), and the routers read those columns alone; it draws routers until every pattern's choice is clear by MARGIN for any
factor from 0.4 to 2.2 that a norm may put on the markers.  The seeds are ones at which rounding the plain implementation's
products to bfloat16 moves no logit by more than about 1.2% of the largest (a norm behind a sublayer makes a small branch large).
"""
import os

import torch

MARKERS = 3            # columns, the last ones
MARK = 2.0
BRANCH = 0.5
MARGIN = 0.02          # of the corrected scores


def _att(heads, kv_heads, dim, scale, window=None, rot=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale}
    if window:
        m["mask"] = {"size": window}
    if rot:
        m["rot"] = dict(zip(("dims", "base"), rot))
    return "attention", m


def _att2(heads, kv_heads, dim, vdim, scale, chunk=None, cap=None, rot=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if chunk:
        m["mask"] = {"size": chunk}
    if cap:
        m["softcap"] = cap
    if rot:
        m["rot"] = dict(zip(("dims", "base"), rot))
    return "attention_2", m


def _ssm(heads, vdim, state, groups, conv, norm_groups):
    return "mamba2", {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(ff, experts, top, identity=0, shared=0):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if identity:
        m["router"]["identity"] = identity
    if shared:
        m["shared"] = {"ff": shared}
    return m


def _config(vocab, width, eps, groups, taps, scale, cap, layers):
    out = {"architecture": "Litizen", "vocab": vocab, "width": width, "norm": {"eps": eps, "groups": groups}, "canon": {"taps": taps},
           "embedding": {"scale": scale}, "layers": [{"type": t, "mixer": m, "mlp": mlp} for (t, m), mlp in layers]}
    if cap:
        out["logit_softcap"] = cap
    return out


MODELS = {
    "A": dict(config=_config(311, 96, 1e-5, 3, 3, 0.7, 12.0, [
        (_att2(6, 2, 16, 24, 0.4, 21, 9.0, (8, 500.0)), _moe(48, 4, 2, 1, 40)),
        (_ssm(4, 20, 12, 2, 4, 5), _dense(128)),
        (_att(6, 2, 16, 0.6, 19, (10, 90.0)), _moe(40, 5, 3, 2)),
        (_ssm(3, 16, 24, 1, 2, 1), None)]),
        seed=71, linear_std=0.1, norm_std=0.15, page_size=16),
    "B": dict(config=_config(257, 100, 1e-6, 1, 1, 1.0, None, [
        (_att(5, 5, 20, 0.5, 1, (20, 1000.0)), _moe(60, 3, 1)),
        (_att2(4, 4, 24, 24, 0.35, 8, None, (24, 200.0)), None),
        (_ssm(1, 40, 40, 1, 1, 1), _dense(100))]),
        seed=52, linear_std=0.1, norm_std=0.2, page_size=8),
    "C": dict(config=_config(131, 50, 1e-5, 5, 6, 1.9, 7.0, [
        (_att(3, 1, 12, 0.7, 3, (6, 40.0)), _moe(22, 5, 8, 3, 18)),
        (_ssm(6, 6, 7, 3, 6, 4), _dense(34)),
        (_att2(3, 1, 20, 10, 0.5, 5, 6.0, (4, 30.0)), _moe(14, 6, 2, 1, 26)),
        (_att2(2, 2, 6, 18, 0.6, 1, 8.0, (6, 60.0)), None)]),
        seed=64, linear_std=0.14, norm_std=0.1, page_size=8),
    "M": dict(config=_config(190, 72, 1e-6, 2, 5, 0.4, 20.0, [
        (_ssm(4, 12, 16, 4, 3, 4), _dense(48)), (_ssm(2, 33, 9, 2, 5, 6), _moe(32, 4, 2, 2, 16)), (_ssm(6, 8, 32, 3, 2, 1), None)]),
        seed=71, linear_std=0.1, norm_std=0.15, page_size=8),
    "R": dict(config=_config(409, 384, 1e-6, 4, 4, 0.6, 25.0, [
        (_att(4, 4, 128, 0.09, 100, (128, 50000.0)), _moe(128, 8, 3, 3, 160)),
        (_ssm(8, 64, 64, 2, 4, 2), _dense(768)),
        (_att2(6, 2, 64, 96, 0.12, 150, 15.0, (32, 20000.0)), _moe(96, 8, 2, 1)),
        (_att2(4, 2, 128, 128, 0.09, 70, 30.0, (64, 9000.0)), None)]),
        seed=55, linear_std=0.05, norm_std=0.1, page_size=64),
    "S": dict(config=_config(300, 320, 1e-5, 2, 2, 1.3, 18.0, [
        (_att2(8, 1, 64, 64, 0.13, 70, 10.0, (48, 5000.0)), _dense(320)),
        (_att(8, 1, 64, 0.2, 1000, (64, 9000.0)), _moe(64, 6, 2, 2, 64)),
        (_att(4, 2, 32, 0.3, None, None), None),
        (_att2(4, 4, 32, 48, 0.2, None, 9.0, (16, 700.0)), _moe(72, 3, 3, 1, 40))]),
        seed=56, linear_std=0.06, norm_std=0.1, page_size=64),
}


def _router(experts, real, top, g):
    """(rows [experts, MARKERS], correction [experts]) whose choice is clear for every pattern of the markers, at every factor; that
    is not the same for all patterns, nor what it would be without the correction, and takes identity experts where there are any."""
    pats = torch.tensor([[1.0 if (p >> b) & 1 else -1.0 for b in range(MARKERS)] for p in range(1 << MARKERS)])
    for _ in range(200000):
        rw = (torch.randn(experts, MARKERS, generator=g) * 0.9).to(torch.bfloat16).float()
        corr = (torch.randn(experts, generator=g) * 0.15).to(torch.bfloat16).float()
        clear, same, plain = True, None, None
        for factor in (0.4, 0.7, 1.0, 1.5, 2.2):
            scores = torch.softmax(factor * pats @ rw.T, dim=-1)
            s = (scores + corr).sort(dim=-1, descending=True)
            chosen = s.indices[:, :top].sort(dim=-1).values
            plain = scores.topk(top, dim=-1).indices.sort(dim=-1).values
            if (top < experts and float((s.values[:, top - 1] - s.values[:, top]).min()) < MARGIN) or (
                    same is not None and not torch.equal(chosen, same)):
                clear = False
                break
            same = chosen
        if clear and (top == experts or (len({tuple(r) for r in same.tolist()}) >= 3 and bool((same != plain).any())
                                         and (experts == real or bool((same >= real).any())))):
            return rw, corr
    raise RuntimeError("no decisive router found")


def make_model(model_dir, name):
    """Writes the folder of configuration `name`: random weights with decisive routers, sinks that matter beside the scores and
    state spaces that reach far back; returns the folder."""
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
    c = t["config"]
    cols = list(range(c["width"] - MARKERS, c["width"]))
    ids = torch.arange(c["vocab"])
    W["embed"] = W["embed"] / W["embed"].float().std() / c["embedding"]["scale"]      # a stream of about 1
    W["embed"] = W["embed"].to(torch.bfloat16)
    for b, col in enumerate(cols):
        W["embed"][:, col] = (((ids >> b) & 1).float() * 2 - 1) * MARK / c["embedding"]["scale"]
    g = torch.Generator().manual_seed(t["seed"])
    for k in W:
        if k.endswith((".norm1b", ".norm2b")):
            # branches below the embedding (their norms would let every layer's rounding in at full size), and nothing but the
            # embedding writes to the marker columns
            W[k] = (W[k].float() * BRANCH).to(torch.bfloat16)
            W[k][cols] = 0
        if k.endswith(".sink"):
            W[k] = (W[k].float() * 2).to(torch.bfloat16)
        if k.endswith(".A_log"):                           # decays from fast to slow
            n = W[k].shape[0]
            W[k] = torch.linspace(-4.0, 0.5, n).to(torch.bfloat16)
    for i, layer in enumerate(c["layers"]):
        ml = layer.get("mlp")
        if not ml or ml["kind"] != "moe":
            continue
        W[f"l{i}.norm2"][cols] = 1.0
        experts, top = ml["router"]["experts"] + ml["router"].get("identity", 0), ml["router"]["top"]
        r = torch.zeros_like(W[f"l{i}.mlp.router"], dtype=torch.float32)
        r[:, cols], corr = _router(experts, ml["router"]["experts"], top, g)
        W[f"l{i}.mlp.correction"] = corr.to(torch.bfloat16)
        W[f"l{i}.mlp.router"] = r.to(torch.bfloat16)
    save_file({k: v.contiguous() for k, v in W.items()}, path)
    return model_dir
