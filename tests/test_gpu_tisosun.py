"""Tisosun on the GPU against the plain implementation (tests/plain_tisosun.py): each mechanism's kernel alone, then whole
models under every way of cutting the work, in float32 and bfloat16."""
import json
import math
import os
import random
import subprocess
import sys

import numpy as np
import pytest
import torch

import harness
import plain_tisosun as plain
from tisosun_models import MODELS, make_model

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
REPO = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = ["float32", "bfloat16"]
TD = {"float32": torch.float32, "bfloat16": torch.bfloat16}
TOL = {"float32": 2e-5, "bfloat16": 2e-2}


@pytest.fixture(scope="module")
def dirs(tmp_path_factory):
    root = tmp_path_factory.mktemp("tisosun")
    made = {}

    def get(name):
        if name not in made:
            made[name] = make_model(str(root / name), name)
        return made[name]
    return get


def _i32(x):
    return torch.tensor(x, dtype=torch.int32, device=DEV)


def _i64(x):
    return torch.tensor(x, dtype=torch.int64, device=DEV)


def _steps(cuts):
    """cuts: for each request the sizes of its portions, one a step.  Yields for every step the rows
    (request, first token, tokens) of the requests that still bring something."""
    at = [0] * len(cuts)
    for step in range(max(len(c) for c in cuts)):
        rows = []
        for b, c in enumerate(cuts):
            if step < len(c):
                rows.append((b, at[b], c[step]))
                at[b] += c[step]
        yield rows


def _cu(rows):
    cu = [0]
    for _, _, n in rows:
        cu.append(cu[-1] + n)
    return cu


# ---- what the stream is still to get ---------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,H", [(3, 50), (7, 96), (300, 100), (5, 1100), (300, 1536), (4, 4096), (3, 6144), (2, 9000), (270, 4100)])
def test_stream_join(T, H, dtype):
    """Terms with and without a norm (rows, and stacks of partial sums), the average over the depth, two norms of the new
    row, a subset of rows: every output against the same sums in float64."""
    from xinfer_amd import kernels
    dt = TD[dtype]
    g = torch.Generator().manual_seed(T + H)
    r = lambda *s: torch.randn(*s, generator=g)
    x, first, past = r(T, H), r(T, H), r(11, T, H)
    plain_rows, stack, n1, n2 = r(T, H).to(dt), r(3, T, H), (r(T, H) * 3).to(dt), r(6, T, H) * 0.3
    w1, w2, v1, v2 = (1 + 0.2 * r(H) for _ in range(4))
    d = lambda t: t.to(DEV)
    terms = {"rows": (plain_rows, None, 0.0, 1.0), "stack": (stack, None, 0.0, 0.7), "normed": (n1, w1, 1e-5, 0.5), "normed stack": (n2, w2, 1e-3, -2.0)}

    def value(t):
        y, w, eps, f = t
        y = y.double() if y.dim() == 2 else y.double().sum(0)
        return f * (y if w is None else plain.rms_norm(y, eps, w.double()))

    def close(a, b, tol):
        assert (a.cpu().double() - b).abs().max() < tol * b.abs().max()
    tol = 5e-6 if dtype == "float32" else 8e-3
    for names, n_past in (((), None), (("rows",), None), (("rows", "stack"), 0), (("normed", "rows"), 1), (("normed", "normed stack", "stack"), 3),
                          (("stack", "normed stack", "normed", "rows"), 11), (("normed",), 8)):
        use = [terms[n] for n in names]
        s = x.double() + sum((value(t) for t in use), torch.zeros(T, H, dtype=torch.float64))
        u, avg = s, None
        if n_past is not None:
            coef = 0.4 * r(n_past + 2) / (n_past + 1)
            u = plain.depth_average(coef.double(), [first.double()] + [p.double() for p in past[:n_past]] + [s])
            avg = (d(first), d(past), n_past, d(coef))
        dev_terms = [(d(y), None if w is None else d(w), eps, f) for y, w, eps, f in use]
        norms = [(d(v1), 1e-5), (d(v2), 1e-2)]
        xd = d(x)
        res, low, new, (h1, h2) = kernels.stream_join(xd, dev_terms, norms, dt, keep=True, rounded=True, average=avg)
        close(res, s, 5e-6)
        close(low, s, tol)
        assert (new is None) == (avg is None)
        if avg is not None:
            close(new, u, 5e-6)
        close(h1, plain.rms_norm(u, 1e-5, v1.double()), tol)
        close(h2, plain.rms_norm(u, 1e-2, v2.double()), tol)
        assert torch.equal(xd.cpu(), x)                                        # the stream's tensor is left alone
        rows = [T - 1, 0, T // 2]
        some = kernels.stream_join(xd, dev_terms, norms[:1], dt, average=avg, rows=_i32(rows))[3][0]
        close(some, plain.rms_norm(u, 1e-5, v1.double())[rows], tol)      # (few rows may run with more threads: other sums)
    zeros = kernels.stream_join(None, [(d(n1), d(w1), 1e-5, 0.5)], keep=True, shape=(T, H))[0]
    close(zeros, value(terms["normed"]), 5e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H", [50, 96, 1000])
def test_a_normed_embedding(H, dtype):
    from xinfer_amd import kernels
    g = torch.Generator().manual_seed(H)
    table, w, ids = torch.randn(40, H, generator=g).to(TD[dtype]), 1 + 0.3 * torch.randn(H, generator=g), [3, 39, 0, 3, 17]
    got = kernels.embed_norm(table.to(DEV), _i32(ids), 1.5, w.to(DEV), 1e-5).cpu().double()
    want = plain.rms_norm(table.double()[ids] * 1.5, 1e-5, w.double())
    assert (got - want).abs().max() < 2e-6 * want.abs().max()


# ---- a layer's own input for the token ----------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,K,dim", [(1, 96, 12), (9, 100, 1), (8, 384, 32), (64, 72, 6), (150, 96, 20), (20, 1000, 128)])
def test_token_input(T, K, dim, dtype):
    """The gate's product inside the kernel (few tokens) and before it, from the middle of a table's row."""
    from xinfer_amd import kernels
    dt = TD[dtype]
    g = torch.Generator().manual_seed(T)
    x, w = torch.randn(T, K, generator=g).to(dt), (torch.randn(dim, K, generator=g) * 2 / K ** 0.5).to(dt)
    table = torch.randn(50, 3 * dim + 5, generator=g).to(dt)
    ids = torch.randint(0, 50, (T,), generator=g)
    z = x.double() @ w.double().T
    want = plain.gelu_tanh(z) * table.double()[ids][:, dim + 2:2 * dim + 2]
    tol = 2e-5 if dtype == "float32" else 1e-2
    zs = torch.stack([z.float() * 0.25, z.float() * 0.75])
    got = kernels.side_mul(zs.to(DEV), table.to(DEV), dim + 2, ids.int().to(DEV)).cpu().double()
    assert (got - want).abs().max() < tol * want.abs().max()
    got = kernels.side_mul(z.to(dt).to(DEV), table.to(DEV), dim + 2, ids.int().to(DEV)).cpu().double()
    assert (got - want).abs().max() < 2 * tol * want.abs().max()
    if kernels.side_gate_takes(T, K, dt):
        got = kernels.side_gate(x.to(DEV), w.to(DEV), table.to(DEV), dim + 2, ids.int().to(DEV)).cpu().double()
        assert (got - want).abs().max() < tol * want.abs().max()


# ---- recurrences of one number a channel ----------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("chunk", [0, 16])
@pytest.mark.parametrize("C", [33, 64, 1030])
def test_channel_recurrences_of_unequal_requests_in_portions(C, chunk, dtype, monkeypatch):
    """Three requests in slots that are not in order and were used before (the runner's part, clearing a slot, is done here by
    hand), cut into portions down to one token; long portions in chunks side by side; both sources of a and b."""
    from xinfer_amd import kernels
    monkeypatch.setattr(kernels, "CHANNEL_CHUNK", chunk)
    dt = TD[dtype]
    lens, cuts, slots = [120, 1, 45], [[2, 99, 1, 18], [1], [40, 1, 1, 3]], [3, 0, 2]
    g = torch.Generator().manual_seed(C)
    packed = [torch.randn(n, 3 * C, generator=g).to(dt) * 2 for n in lens]
    zb, ub, gb = (torch.randn(C, generator=g) for _ in range(3))
    for source in ("mingru", "ready"):
        state = torch.full((5, C), 7.0, device=DEV)
        for s in slots:
            state[s] = 0
        got = [[] for _ in lens]
        ready = [(torch.rand(n, C, generator=g), torch.randn(n, C, generator=g)) for n in lens]
        for rows in _steps(cuts):
            p = torch.cat([packed[r][s:s + n] for r, s, n in rows]).to(DEV)
            kw = (dict(mingru=(p[:, :C], zb.to(DEV), p[:, C:2 * C], ub.to(DEV))) if source == "mingru" else
                  dict(ready=tuple(torch.cat([ready[r][k][s:s + n] for r, s, n in rows]).to(DEV) for k in (0, 1)), gate_bias=gb.to(DEV)))
            out = kernels.channel_scan(p[:, 2 * C:], "silu" if source == "mingru" else "gelu_tanh", state,
                                       _i64([slots[r] for r, _, _ in rows]), _i32(_cu(rows)), q_lens=[n for _, _, n in rows],
                                       plan_cache={}, **kw)
            for i, (r, _, _) in enumerate(rows):
                got[r].append(out[_cu(rows)[i]:_cu(rows)[i + 1]].cpu())
        assert float(state[1].min()) == 7.0 and float(state[4].max()) == 7.0
        for r in range(3):
            p = packed[r].double()
            if source == "mingru":
                a, b = plain.mingru_terms(p[:, :C] + zb.double(), p[:, C:2 * C] + ub.double())
                gate = plain.silu(p[:, 2 * C:])
            else:
                a, b = (t.double() for t in ready[r])
                gate = plain.gelu_tanh(p[:, 2 * C:] + gb.double())
            S, last = plain.channel_recurrence(a, b)
            want = S * gate
            err = (torch.cat(got[r]).double() - want).abs().max(dim=1).values
            bad = (err > (1e-5 if dtype == "float32" else 6e-3) * want.abs().max()).nonzero()
            assert bad.numel() == 0, f"{source}, request {r}: first wrong token {int(bad[0])}"
            assert (state[slots[r]].cpu().double() - last).abs().max() < 1e-5 * last.abs().max()


@pytest.mark.parametrize("far", [900, 299, 40])
def test_channel_recurrence_keeps_a_far_token(far):
    """Gates that shut all but one token out: what that token left is there `far` tokens later, times the product of the
    decays, through single tokens and through chunks."""
    from xinfer_amd import kernels
    C, T = 24, far + 3
    z = torch.full((T, C), -20.0)
    z[2] = 20.0
    z[3:] = -7.0                       # a = 1 - sigmoid(-7) a token
    u = torch.zeros(T, C)
    u[3:] = -90.0                      # the candidates of the others are (nearly) zero
    u[2] = torch.arange(C) + 1.0
    packed = torch.cat([z, u, torch.full((T, C), 30.0)], dim=1)
    keep = (1.0 - 1.0 / (1.0 + math.exp(7.0))) ** (T - 3)
    for cut in ([T], [T - 3, 1, 1, 1], [7] + [1] * (T - 7)):
        state, at = torch.zeros(1, C, device=DEV), 0
        for n in cut:
            p = packed[at:at + n].to(DEV)
            out = kernels.channel_scan(p[:, 2 * C:], "silu", state, _i64([0]), _i32([0, n]), mingru=(p[:, :C], None, p[:, C:2 * C], None),
                                       q_lens=[n], plan_cache={})
            at += n
        want = keep * (torch.arange(C) + 1.5) * 30.0
        assert (out[-1].cpu() - want).abs().max() < 1e-4 * want.abs().max(), f"cut {cut[:4]}"
        assert keep > 0.3


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,blocks,per", [(7, 3, 40), (130, 1, 100), (40, 7, 6), (300, 4, 128), (33, 2, 72), (1, 2, 8), (150, 5, 16)])
def test_gates_of_the_real_gated_unit(T, blocks, per, dtype, monkeypatch):
    """Block-diagonal products and what is made of them; decays so near 1 that 1 - a^2 would cancel."""
    from xinfer_amd import kernels
    dt, C = TD[dtype], blocks * per
    g = torch.Generator().manual_seed(T)
    u = torch.randn(T, C, generator=g).to(dt)
    w = (torch.randn(blocks, 2, per, per, generator=g) * 2 / per ** 0.5).to(dt)
    rb, ib = torch.randn(C, generator=g), torch.randn(C, generator=g)
    lam = torch.randn(C, generator=g) * 4 - 6
    lam[0] = -16.0
    rate = (-8.0 * plain.softplus(lam.double())).float()
    r = plain.block_gate(u.double(), w[:, 0].double(), rb.double().view(blocks, per))
    i = plain.block_gate(u.double(), w[:, 1].double(), ib.double().view(blocks, per))
    want_a, want_b = plain.rglru_terms(u.double(), r, i, lam.double())
    for matrix_cores in ((True, False) if dtype == "bfloat16" else (False,)):
        monkeypatch.setattr(kernels, "RGLRU_MFMA", matrix_cores)
        a, b = (t.cpu().double() for t in kernels.rglru_terms(u.to(DEV), w.to(DEV), rb.to(DEV), ib.to(DEV), rate.to(DEV)))
        assert ((1 - a) - (1 - want_a)).abs().max() < 2e-5
        rel = ((b - want_b).abs() / (want_b.abs() + 1e-6 * want_b.abs().max())).max()
        assert rel < 1e-2, f"matrix cores {matrix_cores}: {float(rel):.2e}"          # element by element, the tiny ones too
        assert (b - want_b).abs().max() < 2e-5 * want_b.abs().max()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("C,taps", [(120, 3), (100, 1), (42, 6), (64, 4), (512, 4), (80, 2)])
def test_convolution_without_an_activation_behind_a_bias(C, taps, dtype):
    """Portions shorter than the taps, beside another request's tail; the inputs' bias is added to inputs only, not to the
    zeros before a sequence."""
    from xinfer_amd import kernels
    dt = TD[dtype]
    L = 61
    g = torch.Generator().manual_seed(C)
    packed = torch.randn(L, C + 8, generator=g).to(dt)
    w, b, ib = torch.randn(C, taps, generator=g), torch.randn(C, generator=g), torch.randn(C, generator=g) * 2
    want = plain.short_conv(packed[:, 8:].double() + ib.double(), w.double(), b.double())
    tails = torch.full((3, taps - 1, C), 5.0, device=DEV)
    if taps > 1:
        tails[1] = 0
    outs, at = [], 0
    for n in (1, 1, 3, 2, 20, 1, 33):
        rows = packed[at:at + n].to(DEV)[:, 8:]
        outs.append(kernels.causal_conv(rows, w.to(DEV), b.to(DEV), tails, _i64([1]), _i32([0] * n), _i32([0, n]), in_bias=ib.to(DEV),
                                        act="none").cpu())
        if taps > 1:
            kernels.conv_tail(rows, tails, _i64([1]), _i32([0, n]), in_bias=ib.to(DEV))
        at += n
    got = torch.cat(outs).double()
    assert (got - want).abs().max() < (1e-5 if dtype == "float32" else 6e-3) * want.abs().max()
    if taps > 1:
        assert float(tails[0].min()) == 5.0 and float(tails[2].max()) == 5.0
        assert (tails[1].cpu().double() - (packed[L - taps + 1:, 8:].double() + ib.double())).abs().max() < 1e-5


# ---- linear attention behind silu, heads normed together -----------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("chunk", [0, 16, 64])
@pytest.mark.parametrize("H,dk,dv", [(3, 12, 20), (1, 20, 20), (5, 6, 10), (2, 64, 96), (3, 40, 136), (2, 136, 24), (1, 256, 264), (4, 16, 1000)])
def test_lightning_attention_in_portions(H, dk, dv, chunk, dtype, monkeypatch):
    """Token by token, in chunks of the walk, and (bfloat16, sizes in eights) in chunks on the matrix cores, whose last one may
    be a single token; short portions beside long ones; decays from a half to one."""
    from xinfer_amd import kernels
    monkeypatch.setattr(kernels, "SCAN_CHUNK", chunk)
    dt, eps = TD[dtype], 1e-5
    lens, cuts, slots = [170, 1, 45, 64], [[2, 164, 1, 3], [1], [40, 1, 1, 3], [31, 33]], [3, 0, 2, 4]
    g = torch.Generator().manual_seed(H * dk)
    a, b = H * dk, H * dv
    packed = [(torch.randn(n, 2 * a + 2 * b, generator=g)).to(dt) for n in lens]
    decay = torch.linspace(0.5, 1.0, H) if H > 1 else torch.tensor([0.97])
    w = 1 + 0.2 * torch.randn(b, generator=g)
    state = torch.full((6, H, dk, dv), 7.0, device=DEV)
    for s in slots:
        state[s] = 0
    got = [[] for _ in lens]
    for rows in _steps(cuts):
        p = torch.cat([packed[r][s:s + n] for r, s, n in rows]).to(DEV)
        o = kernels.linear_scan(p[:, :a], p[:, a:2 * a], p[:, 2 * a:2 * a + b], state, _i64([slots[r] for r, _, _ in rows]), _i32(_cu(rows)),
                                H, dk, dv, head_decay=decay.to(DEV), silu=True, q_lens=[n for _, _, n in rows], plan_cache={})
        out = kernels.row_norm_gate(o.view(-1, b), w.to(DEV), eps, p[:, 2 * a + b:], "sigmoid")
        for i, (r, _, _) in enumerate(rows):
            got[r].append(out[_cu(rows)[i]:_cu(rows)[i + 1]].cpu())
    assert float(state[1].min()) == 7.0 and float(state[5].max()) == 7.0
    rounded = dtype == "bfloat16" and chunk > 0            # q, k and v behind silu are rounded once on the matrix cores
    for r, n in enumerate(lens):
        p = packed[r].double()
        q, k, v = (plain.silu(t) for t in (p[:, :a].view(n, H, dk), p[:, a:2 * a].view(n, H, dk), p[:, 2 * a:2 * a + b].view(n, H, dv)))
        o, S = plain.decayed_state(q, k, v, [float(x) for x in decay])
        want = plain.rms_norm(o.reshape(n, b), eps, w.double()) * torch.sigmoid(p[:, 2 * a + b:])
        err = (torch.cat(got[r]).double() - want).abs().max(dim=1).values
        bad = (err > (2e-5 if dtype == "float32" else 1.2e-2) * want.abs().max()).nonzero()
        assert bad.numel() == 0, f"request {r}: first wrong token {int(bad[0])}: {float(err[int(bad[0])]):.2e} of {float(want.abs().max()):.2e}"
        assert (state[slots[r]].cpu().double() - S).abs().max() < (4e-3 if rounded else 2e-5) * max(1.0, float(S.abs().max()))


@pytest.mark.parametrize("H,dk,dv,silu", [(2, 64, 40, False), (3, 32, 128, True), (1, 128, 64, False)])
def test_decayed_states_on_the_matrix_cores_keep_float32(H, dk, dv, silu, monkeypatch):
    """Inputs that bfloat16 holds exactly: the chunks' results and states then agree with the plain walk far below
    bfloat16's rounding, whatever decays multiply in between, and a key planted hundreds of tokens back is read."""
    from xinfer_amd import kernels
    T, a = 700, H * dk
    g = torch.Generator().manual_seed(dk)
    p = torch.randn(T, 2 * a + H * dv, generator=g) * 0.5
    p[3, a:2 * a] = 6.0                                    # token 3's key and value stand out
    p[3, 2 * a:] = 8.0
    p = p.bfloat16()
    decay = torch.tensor([0.9973, 0.62, 0.99991][:H])
    act = (lambda t: plain.silu(t).bfloat16().double()) if silu else (lambda t: t)
    q, k, v = (act(t) for t in (p[:, :a].double().view(T, H, dk), p[:, a:2 * a].double().view(T, H, dk), p[:, 2 * a:].double().view(T, H, dv)))
    want, S = plain.decayed_state(q, 0.25 * k, v, [float(d) for d in decay])
    state = torch.zeros(2, H, dk, dv, device=DEV)
    outs, at = [], 0
    for n in (40, 1, 459, 200):
        rows = p[at:at + n].to(DEV)
        outs.append(kernels.linear_scan(rows[:, :a], rows[:, a:2 * a], rows[:, 2 * a:], state, _i64([1]), _i32([0, n]), H, dk, dv,
                                        head_decay=decay.to(DEV), k_scale=0.25, silu=silu, q_lens=[n], plan_cache={}).cpu())
        at += n
    got = torch.cat(outs).double()
    tol = 3e-3 if silu else 3e-5            # (silu: the single token's walk does not round it, and the hardware's last bits move roundings)
    assert (got - want).abs().max() < tol * want.abs().max()
    assert (state[1].cpu().double() - S).abs().max() < tol * S.abs().max()
    assert float(state[0].abs().max()) == 0


def test_rows_normed_together_and_gated():
    from xinfer_amd import kernels
    g = torch.Generator().manual_seed(5)
    for T, W in ((3, 50), (300, 48), (2, 4096), (260, 5000), (1, 20000)):
        o, w, gate = torch.randn(T, W, generator=g) * 2, torch.randn(W, generator=g), torch.randn(T, W + 8, generator=g)
        n = plain.rms_norm(o.double(), 1e-5, w.double())
        for act, f in (("sigmoid", torch.sigmoid), ("silu", plain.silu)):
            got = kernels.row_norm_gate(o.to(DEV), w.to(DEV), 1e-5, gate.to(DEV)[:, 8:], act).cpu().double()
            want = n * f(gate[:, 8:].double())
            assert (got - want).abs().max() < 5e-6 * want.abs().max()


# ---- attention within chunks ---------------------------------------------------------------------------------------------
def _pools(L, G, d, dv, page, dtype, grouped, seed=0):
    """Empty K and V pools with more pages than L tokens need, and a block table of shuffled pages."""
    n_pages = -(-L // page)
    order = list(range(n_pages + 3))
    random.Random(seed).shuffle(order)
    table = torch.tensor([order[:n_pages]], dtype=torch.int32)
    k_pool = torch.zeros((n_pages + 3, G, page, d), dtype=dtype)
    v_pool = torch.zeros((n_pages + 3, G, page // 8, dv, 8) if grouped else (n_pages + 3, G, page, dv), dtype=dtype)
    slots = torch.tensor([order[p // page] * page + p % page for p in range(L)], dtype=torch.int64)
    return k_pool, v_pool, table, slots


def _read_pools(k_pool, v_pool, table, L, grouped):
    page = k_pool.shape[2]
    k = torch.stack([k_pool[table[0, p // page], :, p % page] for p in range(L)])
    v = torch.stack([v_pool[table[0, p // page], :, (p % page) // 8, :, p % 8] if grouped else v_pool[table[0, p // page], :, p % page]
                     for p in range(L)])
    return k, v


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("L", [45, 301])
@pytest.mark.parametrize("H,G,d,dv,rot,page,norms", [(6, 2, 16, 24, 8, 16, True), (2, 2, 128, 40, 64, 16, True), (3, 1, 24, 256, 12, 8, True), (5, 5, 20, 12, 20, 8, True), (3, 1, 12, 20, 6, 8, True),
                                                     (2, 1, 10, 6, 0, 8, True), (4, 2, 64, 48, 32, 64, True), (3, 3, 16, 8, 16, 8, False)])
def test_heads_with_biases_norms_and_turned_pairs(H, G, d, dv, rot, page, norms, L, dtype):
    """Bias, norm with a weight, rotation of the pairs (2i, 2i + 1) in that order, and the cache write, a head a wave and (many
    tokens, sizes in eights) eight dims a lane."""
    from xinfer_amd import kernels
    dt, eps = TD[dtype], 1e-5
    grouped = dtype == "bfloat16"
    g = torch.Generator().manual_seed(H * 10 + d)
    width = (H + G) * d + G * dv
    packed, bias = torch.randn(L, width, generator=g).to(dt), torch.randn(width, generator=g)
    qw, kw = (1 + 0.3 * torch.randn(d, generator=g), 1 + 0.3 * torch.randn(d, generator=g)) if norms else (None, None)
    full = packed.double() + bias.double()
    q, k, v = full[:, :H * d].view(L, H, d), full[:, H * d:(H + G) * d].view(L, G, d), full[:, (H + G) * d:].view(L, G, dv)
    if norms:
        q, k = plain.rms_norm(q, eps, qw.double()), plain.rms_norm(k, eps, kw.double())
    r = dict(dims=rot, base=90.0, scaling=dict(factor=3.0, original=40, fast=5.0, slow=1.0)) if rot else None
    kwargs = {}
    if rot:
        f, grow = plain.rotary_frequencies(r)
        ang = torch.arange(L, dtype=torch.float64)[:, None] * f
        kwargs = dict(cos=(ang.cos() * grow).float().to(DEV), sin=(ang.sin() * grow).float().to(DEV), rotary_dim=rot, interleaved=True)
        q, k = plain.rotate_pairs(q, r, torch.arange(L)), plain.rotate_pairs(k, r, torch.arange(L))
    k_pool, v_pool, table, slots = _pools(L, G, d, dv, page, dt, grouped, seed=d)
    k_pool, v_pool = k_pool.to(DEV), v_pool.to(DEV)
    slots[5] = -1                                                             # a token that stores nothing
    got = kernels.head_rows(packed.to(DEV), slots.to(DEV), k_pool, v_pool, H, G, d, dv, v_grouped=grouped, positions=_i32(list(range(L))),
                            eps=eps, bias=bias.to(DEV), q_weight=None if qw is None else qw.to(DEV),
                            k_weight=None if kw is None else kw.to(DEV), **kwargs)
    tol = 1e-5 if dtype == "float32" else 6e-3
    assert (got.cpu().double() - q).abs().max() < tol * q.abs().max()
    gk, gv = _read_pools(k_pool.cpu(), v_pool.cpu(), table, L, grouped)
    keep = [p for p in range(L) if p != 5]
    assert (gk.double()[keep] - k[keep]).abs().max() < tol * k.abs().max() and (gv.double()[keep] - v[keep]).abs().max() < tol * v.abs().max()
    assert float(gk[5].abs().max()) == 0 and float(gv[5].abs().max()) == 0


def _planted(L, H, G, d, chunk, scale, seed):
    """q [L, H, d] and k [L, G, d] in which chosen (query, key) pairs have a score that stands far out: keys just inside and just
    outside a chunk's edges, at page borders, at the first tokens, far back."""
    g = torch.Generator().manual_seed(seed)
    q = torch.randn(L, H, d, generator=g) * 0.3
    k = torch.randn(L, G, d, generator=g) * 0.3
    big = 30.0 / scale
    c = chunk or L
    queries = set(range(max(0, L - 12), L)) | {1, 2, 17, 31, 32, 63, 64, 65, 128} | {e + o for e in range(0, L, c) for o in (-1, 0, 1, 2)}
    pairs = []
    for i in sorted(queries):
        if not (0 <= i < L):
            continue
        edge = i - i % c
        for j in (i, i - 1, edge, edge + 1, edge - 1, edge - 2, i - 15, i - 16, i - 64, 0, 1, edge - c, i - L + 3):
            if 0 <= j <= i:
                pairs.append((i, j))
    rng = random.Random(seed)
    rng.shuffle(pairs)
    for n, (i, j) in enumerate(pairs):
        h = rng.randrange(H)
        u = torch.zeros(d)
        u[n % d] = big ** 0.5
        q[i, h] = u
        k[j, h // (H // G)] = u
    return q, k


CHUNK_CASES = [  # H, G, d, dv, chunk, cap, scale, L, page
    (6, 2, 16, 24, 21, 15.0, 0.4, 90, 16),
    (5, 5, 24, 24, 8, 0.0, 0.3, 70, 8),
    (3, 1, 16, 24, 5, 20.0, 0.5, 61, 8),
    (3, 1, 12, 20, 7, 20.0, 0.5, 61, 8),          # sizes that the matrix-core kernel does not take
    (2, 2, 16, 8, 1, 0.0, 0.5, 40, 8),
    (8, 2, 64, 48, 100, 25.0, 0.11, 330, 64),
    (4, 2, 128, 128, 150, 40.0, 0.09, 400, 64),
    (8, 1, 64, 96, 70, 30.0, 0.12, 300, 64),       # single tokens: the heads are the rows of a block
    (4, 4, 32, 64, 64, 0.0, 0.2, 200, 32),
    (8, 1, 64, 64, 500, 0.0, 0.12, 260, 64),        # chunks wider than the request
    (6, 3, 200, 40, 33, 12.0, 0.1, 120, 16),
    (4, 2, 32, 32, 0, 9.0, 0.2, 150, 16),           # no chunks
]


def _chunk_case(case, dtype, matrix_cores, tail):
    from xinfer_amd import kernels
    H, G, d, dv, chunk, cap, scale, L, page = case
    dt, grouped = TD[dtype], dtype == "bfloat16"
    q, k = _planted(L, H, G, d, chunk, scale, seed=L)
    v = torch.randn(L, G, dv, generator=torch.Generator().manual_seed(L))
    q, k, v = q.to(dt), k.to(dt), v.to(dt)
    want = plain.softmax_heads(q.double(), k.double(), v.double(), scale, cap, chunk)
    if 0 < chunk < L:                                                              # where the edges lie matters here
        for other in (chunk + 1, max(1, chunk - 1), 0):
            if other != chunk:
                assert (plain.softmax_heads(q.double(), k.double(), v.double(), scale, cap, other) - want).abs().max() > 0.1 * want.abs().max()
    k_pool, v_pool, table, slots = _pools(L, G, d, dv, page, dt, grouped, seed=L)
    for p in range(L):
        pg, off = int(slots[p]) // page, int(slots[p]) % page
        k_pool[pg, :, off] = k[p]
        if grouped:
            v_pool[pg, :, off // 8, :, off % 8] = v[p]
        else:
            v_pool[pg, :, off] = v[p]
    k_pool, v_pool, table = k_pool.to(DEV), v_pool.to(DEV), table.to(DEV)

    def run(positions):
        qs, pos = q[positions[0]:positions[-1] + 1].to(DEV), _i32(positions)
        if not matrix_cores:
            return kernels.attention_generic(qs, k_pool, v_pool, table, torch.zeros_like(pos), pos, scale, 0, v_grouped=grouped, softcap=cap,
                                             chunk=chunk)
        n, ctx = len(positions), positions[-1] + 1
        span = min(ctx, chunk + 63) if chunk else ctx
        if n == 1 and G == 1 and H >= 4 and positions[0] % 3:        # a token's heads as the rows of a block
            shape = 1 if kernels.attention_biased_block(d, dv, 1, 1) >= H else 0
            per = kernels.attention_biased_block(d, dv, 1, shape)
            tiles = _i32([[0, i * per] for i in range(-(-H // per))])
            return kernels.attention_biased_bf16(qs.view(H, 1, d), k_pool, v_pool, table, tiles, _i32([0, H]), _i32([ctx]), scale, 0,
                                                 softcap=cap, small=shape, split_keys=64 if positions[0] % 2 else 0, span=span,
                                                 rows_heads=H, chunk=chunk).view(1, H * dv)
        rows, shape = kernels.prefill_tiles([n], [ctx], d, H, G, block_of=lambda s_: kernels.attention_biased_block(d, dv, H // G, s_))
        tiles = torch.tensor(rows, dtype=torch.int32, device=DEV).reshape(-1, 2)
        split = 64 if n == 1 and positions[0] % 2 else 0              # every other single token in slices of 64 keys
        return kernels.attention_biased_bf16(qs, k_pool, v_pool, table, tiles, _i32([0, n]), _i32([ctx]), scale, 0, softcap=cap, small=shape,
                                             split_keys=split, span=span if split else 0, chunk=chunk)
    head = max(1, L - tail)
    cuts = [0, head // 3 + 1, head] if head > 8 else [0, head]
    outs = [run(list(range(a, b))) for a, b in zip(cuts[:-1], cuts[1:]) if b > a] + [run([p]) for p in range(head, L)]
    got = torch.cat([o.cpu() for o in outs]).double()
    err = (got - want).abs().max(dim=1).values
    bad = (err > TOL[dtype] * want.abs().max()).nonzero()
    assert bad.numel() == 0, f"first wrong position {int(bad[0])} of {L} (chunks of {chunk}): {float(err[int(bad[0])]):.3e}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", CHUNK_CASES)
def test_attention_within_chunks_with_planted_keys(case, dtype):
    _chunk_case(case, dtype, matrix_cores=False, tail=9)


@pytest.mark.parametrize("case", [c for c in CHUNK_CASES if c[2] % 8 == 0 and c[3] % 8 == 0])
def test_attention_within_chunks_on_the_matrix_cores(case):
    _chunk_case(case, "bfloat16", matrix_cores=True, tail=9)
    _chunk_case(case, "bfloat16", matrix_cores=True, tail=75)


# ---- whole models ----------------------------------------------------------------------------------------------------
LENGTHS = {"A": [1, 2, 21, 22, 43, 77, 130], "B": [3, 8, 9, 18, 64, 101], "C": [1, 5, 6, 40, 75, 210], "M": [2, 1, 30, 140],
           "R": [5, 101, 330, 64, 301], "S": [3, 70, 71, 260, 129]}


def _requests(name):
    rng = random.Random(700 + ord(name))
    vocab = MODELS[name]["config"]["vocab"]
    return {f"r{i}": harness.random_prompt(rng, n, vocab) for i, n in enumerate(LENGTHS[name])}


_plain_cache = {}
_model_cache = {}


def _plain_logits(name, model_dir):
    if name not in _plain_cache:
        pm = plain.PlainTisosun(model_dir, torch.float64)
        _plain_cache[name] = {rid: pm.logits(toks).float() for rid, toks in _requests(name).items()}
    return _plain_cache[name]


def _model(name, dtype, model_dir):
    from xinfer_amd.engine import load_model
    if (name, dtype) not in _model_cache:
        _model_cache[(name, dtype)] = load_model(model_dir, dtype, DEV)
    return _model_cache[(name, dtype)]


def _run(name, dtype, dirs, steps, what, **kw):
    from xinfer_amd.engine import ModelRunner
    page = MODELS[name]["page_size"]
    need = harness.tokens_needed(steps, page)
    model = _model(name, dtype, dirs(name))
    runner = ModelRunner(model, page_size=page, num_pages=max(1, need // page), max_requests=4, **kw)     # exactly enough pages
    got = harness.replay(runner, steps)
    for g in range(len(runner.cache.groups)):
        assert runner.cache.free_pages(g) == max(1, need // page)
    rel = harness.compare(got, _plain_logits(name, dirs(name)), harness.TOL[dtype], f"{name}/{dtype}/{what}")
    print(f"{name}/{dtype}/{what}: worst error {rel:.2e} of the largest logit")
    return got, runner


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MODELS))
def test_whole(name, dtype, dirs):
    got, _ = _run(name, dtype, dirs, harness.trace_whole(_requests(name)), "whole")
    assert len(got) == sum(LENGTHS[name])


@pytest.mark.parametrize("name", ["A", "B", "C", "M"])
def test_the_stream_after_every_layer(name, dirs):
    """float32, one request: what every layer hands on, and its own result before the average, against the plain ones."""
    from xinfer_amd.engine import ModelRunner, StepEntry
    from xinfer_amd.parts.joining import join
    model = _model(name, "float32", dirs(name))
    toks = _requests(name)["r2"]
    pm = plain.PlainTisosun(dirs(name), torch.float64)
    want, results = pm.stream(toks)[1:], pm.stream(toks, averaged=False)[1:]
    seen = []
    last = [model.stream_ops[id(e.after[-1])] for e in model.spec.schedule]
    kept = [(op, op.forward) for op in last]
    try:
        for op, orig in kept:
            def fwd(stream, first, ctx, _o=orig):
                s = _o(stream, first, ctx)
                seen.append((join(s, torch.float32)[0].resid.cpu().double(), s.average.results[s.average.place].cpu().double()))
                return s
            op.forward = fwd
        runner = ModelRunner(model, page_size=MODELS[name]["page_size"], num_pages=8, max_requests=1, use_graphs=False)
        runner.add_request(0)
        runner.step([StepEntry(0, toks, [])])
    finally:
        for op, orig in kept:
            op.forward = orig
    assert len(seen) == len(want)
    for i, (a, b, c) in enumerate(zip(seen, want, results)):
        assert (a[0] - b).abs().max() < 2e-5 * b.abs().max() and (a[1] - c).abs().max() < 2e-5 * c.abs().max(), f"layer {i}"


@pytest.mark.parametrize("dtype", DTYPES)
def test_branches_side_by_side_normed_and_added(dtype, dirs):
    """What the mixer hands on one by one is what it gives as one sum."""
    from xinfer_amd.engine import ModelRunner, StepEntry
    model = _model("A", dtype, dirs("A"))
    mixer = model.blocks[1].mixer
    seen, orig = [], mixer.forward_terms

    def both(x, ctx, cache):
        state = cache.state.clone()
        mixer.forward_terms = orig
        seen.append(mixer.forward(x, ctx, cache).cpu().double())
        cache.state.copy_(state)
        terms = orig(x, ctx, cache)
        seen.append(sum(t.scale * plain.rms_norm((t.y if t.y.dim() == 2 else t.y.sum(0)).cpu().double(), t.eps, t.weight.cpu().double()) for t in terms))
        return terms
    mixer.forward_terms = both
    try:
        runner = ModelRunner(model, page_size=16, num_pages=8, max_requests=1, use_graphs=False)
        runner.add_request(0)
        runner.step([StepEntry(0, _requests("A")["r4"], [])])
    finally:
        del mixer.forward_terms
    assert len(seen) == 2 and (seen[0] - seen[1]).abs().max() < 5e-6 * seen[1].abs().max()


def test_a_block_of_another_arrangement_behind_an_open_stream(dirs):
    """A layer of this family followed by a pre-norm layer that knows nothing of open streams: it is given a joined one."""
    from dataclasses import replace
    from xinfer_amd.engine import build_model
    from xinfer_amd.engine.model import CausalLM
    from xinfer_amd.engine import ModelRunner, StepEntry
    from xinfer_amd.models import config_from_dict
    from xinfer_amd.weights.store import SafetensorsStore
    fam, cfg = config_from_dict(MODELS["A"]["config"])
    spec = fam.spec(cfg)
    layers = list(spec.layers)
    layers[1] = replace(layers[1], block="prenorm")
    spec = replace(spec, layers=tuple(layers))
    model = CausalLM(spec, torch.float32).load(SafetensorsStore(dirs("A")), DEV)
    assert model._copy_first
    runner = ModelRunner(model, page_size=16, num_pages=8, max_requests=1, use_graphs=False)
    runner.add_request(0)
    toks = _requests("A")["r4"]
    got = runner.step([StepEntry(0, toks, list(range(len(toks))))]).cpu().double()

    class PreNormOne(plain.PlainTisosun):
        def logits(self, tokens):
            tok, eps, dim = torch.tensor(tokens), self.cfg["norm"]["eps"], self.cfg["token_side"]["dim"]
            lw = lambda n: plain.layer_norm_weight(self.w[n])
            x = plain.rms_norm(self.w["embed"][tok], eps, lw("embed.norm"))
            results, pos = [x], torch.arange(len(tokens))
            for i, l in enumerate(self.cfg["layers"]):
                m = self.mixer(i, plain.rms_norm(x, eps, lw(f"l{i}.norm1")), pos)
                y = x + m
                if l["mlp"] is not None:
                    of = y if i == 1 else x
                    y = y + plain.dense_mlp(plain.rms_norm(of, eps, lw(f"l{i}.norm2")), plain.sub(self.w, f"l{i}.mlp."))
                y = y + plain.token_side(y, self.w["side.embed"][tok][:, i * dim:(i + 1) * dim], plain.sub(self.w, f"l{i}.side."), eps)
                results.append(y)
                x = plain.depth_average(self.w[f"l{i}.dwa"], results)
            return plain.rms_norm(x, eps, lw("final.norm")) @ self.w["head"].T
    want = PreNormOne(dirs("A"), torch.float64).logits(toks)
    assert (got - want).abs().max() < 2e-5 * want.abs().max()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MODELS))
def test_prefill_against_decoding_one_by_one(name, dtype, dirs):
    _run(name, dtype, dirs, harness.trace_tail_one_by_one(_requests(name), tail=40), "tail")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MODELS))
def test_portions(name, dtype, dirs):
    _run(name, dtype, dirs, harness.trace_portions(_requests(name)), "portions")
    _run(name, dtype, dirs, harness.trace_portions(_requests(name), sizes=(2, 2, 3, 40, 2, 5)), "small portions")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MODELS))
def test_mixed_batches_with_pages_and_slots_used_again(name, dtype, dirs):
    """More requests than state slots, one after the other in the same slots and pages: a request that starts
    finds no state and no convolution inputs of the one before."""
    for seed in (1, 2):
        _run(name, dtype, dirs, harness.trace_mixed(_requests(name), seed, max_live=3), f"mixed {seed}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "R", "M"])
def test_short_chunks_of_the_states_walks(name, dtype, dirs, monkeypatch):
    """Portions from 32 tokens on are walked in chunks of 16: whole prompts, portions and mixed batches again."""
    from xinfer_amd import kernels
    monkeypatch.setattr(kernels, "SCAN_CHUNK", 16)
    monkeypatch.setattr(kernels, "CHANNEL_CHUNK", 16)
    _run(name, dtype, dirs, harness.trace_whole(_requests(name)), "whole, chunks of 16")
    _run(name, dtype, dirs, harness.trace_portions(_requests(name), sizes=(33, 2, 47, 32, 5)), "portions, chunks of 16")
    _run(name, dtype, dirs, harness.trace_mixed(_requests(name), 3, max_live=3, sizes=(40, 2, 35, 64)), "mixed, chunks of 16")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B", "R", "S"])
def test_unequal_requests_decoding_together(name, dtype, dirs):
    reqs = {k: v for k, v in _requests(name).items() if len(v) > 8}
    reqs = dict(list(reqs.items())[:4])
    _run(name, dtype, dirs, harness.trace_batch_decode(reqs, tail=7), "batch decode", use_graphs=False)
    got, runner = _run(name, dtype, dirs, harness.trace_batch_decode(reqs, tail=7), "batch decode, graphs", graph_after=1)
    assert runner.graph_replays > 0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "R"])
def test_long_decoding(name, dtype, dirs):
    """Three tokens of prompt, then the rest one by one: the states and the convolutions' inputs move on token by token,
    and every chunk ends and the next one starts under decoding, over several pages."""
    n = 253 if name == "A" else 340
    toks = harness.random_prompt(random.Random(9), n, MODELS[name]["config"]["vocab"])
    from xinfer_amd.engine import ModelRunner
    ref = {"a": plain.PlainTisosun(dirs(name), torch.float64).logits(toks).float()}
    steps = harness.trace_tail_one_by_one({"a": toks}, tail=n - 3)
    page = MODELS[name]["page_size"]
    runner = ModelRunner(_model(name, dtype, dirs(name)), page_size=page, num_pages=-(-n // page) + 1, max_requests=2, graph_after=2)
    got = harness.replay(runner, steps)
    assert runner.graph_replays > 200
    harness.compare(got, ref, harness.TOL[dtype], f"long decoding {name} {dtype}")


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
def test_greedy_generation_through_the_engine(dtype, dirs):
    """The framework's own entry point and scheduler: five prompts, three at a time, prompts cut into
    portions of 16 tokens, greedy tokens against the plain implementation."""
    from xinfer_amd import Engine, EngineConfig, SamplingParams
    name = "A"
    rng = random.Random(3)
    vocab = MODELS[name]["config"]["vocab"]
    prompts = [harness.random_prompt(rng, n, vocab) for n in (5, 40, 17, 33, 2)]
    eng = Engine(EngineConfig(weight_path=dirs(name), page_size=16, num_pages=24, max_num_seqs=3, prefill_chunk_size=16,
                              max_model_len=128, seed=1), dtype)
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=24, ignore_eos=True))
    pm = plain.PlainTisosun(dirs(name), torch.float64)
    for p, o in zip(prompts, outs):
        assert o.prompt_length == len(p) and o.decoded_length == 24
        if dtype == "f32":
            assert o.token_ids == pm.greedy(p, 24)
        else:
            ids = list(p)
            for t in o.token_ids:
                lg = pm.logits(ids)[-1]
                assert float(lg.max() - lg[t]) <= 2 * harness.TOL["bfloat16"] * float(lg.abs().max())
                ids.append(t)
    assert eng.runner.cache.live_requests() == 0


def test_command_line_runs_the_model(dirs, capsys):
    from xinfer_amd import cli
    rc = cli.main(["--w", dirs("A"), "--prompt-ids", "1,2,3,4,5,6,7,8,9", "--max-tokens", "4", "--max-model-len", "256",
                   "--temperature", "0", "--ignore-eos", "--page-size", "16", "--max-num-seqs", "4", "--dtype", "bf16"])
    assert rc == 0 and "Decoded tokens: 4 in" in capsys.readouterr().out
    rc = cli.main(["--w", dirs("M"), "--prompt-ids", "1,2,3|4,5,6,7", "--max-tokens", "5", "--max-model-len", "64",
                   "--temperature", "0", "--ignore-eos", "--page-size", "8", "--num-pages", "16", "--dtype", "f32"])
    assert rc == 0 and "Decoded tokens: 10 in" in capsys.readouterr().out


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_run_program(dtype, dirs, tmp_path):
    name = "R"
    vocab = MODELS[name]["config"]["vocab"]
    reqs = {f"r{i}": harness.random_prompt(random.Random(60 + i), n, vocab) for i, n in enumerate([33, 170, 5, 64, 200, 9])}
    steps = harness.trace_mixed(reqs, 4)
    need = harness.tokens_needed(steps, 64)
    out = tmp_path / "out"
    proc = subprocess.Popen(
        [sys.executable, os.path.join(REPO, "bin", "trace_run"), "--model", dirs(name), "--dtype", dtype,
         "--out", str(out), "--max-tokens", str(need)],
        stdin=subprocess.PIPE, stdout=subprocess.PIPE, text=True)
    for st in steps:
        proc.stdin.write(json.dumps(st) + "\n")
        proc.stdin.flush()
        assert proc.stdout.readline().strip() == f"done {st['step']}"
    proc.stdin.close()
    assert proc.wait(timeout=120) == 0
    pm = plain.PlainTisosun(dirs(name), torch.float64)
    ref = {rid: pm.logits(t).float() for rid, t in reqs.items()}
    got, fed = {}, {rid: 0 for rid in reqs}
    for st in steps:
        wanted = sum(len(e["want"]) for e in st["entries"])
        arr = np.fromfile(out / f"{st['step']}.f32", dtype="<f4").reshape(wanted, vocab)
        row = 0
        for e in st["entries"]:
            for w in e["want"]:
                got[(e["id"], fed[e["id"]] + w)] = torch.from_numpy(arr[row].copy())
                row += 1
            fed[e["id"]] += len(e["tokens"])
    assert len(got) == sum(len(t) for t in reqs.values())
    harness.compare(got, ref, harness.TOL[dtype], f"trace_run {dtype}")


def test_decode_graph_replays_equal_launches(dirs):
    """float32: steps replayed from a recorded graph give the bits of the same steps launched one by one (the states
    and the convolution's inputs are advanced once a step, in the step that records too)."""
    from xinfer_amd.engine import ModelRunner, StepEntry
    name = "A"
    model = _model(name, "float32", dirs(name))
    vocab, page = MODELS[name]["config"]["vocab"], MODELS[name]["page_size"]
    rng = random.Random(21)
    prompts = {i: harness.random_prompt(rng, rng.randrange(3, 50), vocab) for i in range(4)}
    feed = {i: harness.random_prompt(rng, 30, vocab) for i in prompts}

    def run(use_graphs):
        runner = ModelRunner(model, page, 24, 4, use_graphs=use_graphs, graph_after=1)
        out = []
        for i in prompts:
            runner.add_request(i)
            runner.step([StepEntry(i, prompts[i], [])])
        for step in range(30):
            out.append(runner.step([StepEntry(i, [feed[i][step]], [0]) for i in prompts]).cpu())
        return out, runner
    want, _ = run(False)
    got, r1 = run(True)
    assert r1.graph_replays >= 25
    for k, (a, b) in enumerate(zip(want, got)):
        assert torch.equal(a, b), f"step {k} differs between graph and launches"
