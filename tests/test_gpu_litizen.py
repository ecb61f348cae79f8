"""Litizen on the GPU against the plain implementation (tests/plain_litizen.py): each mechanism's kernel alone, then whole
models under every way of cutting the work, in float32 and bfloat16."""
import json
import os
import random
import subprocess
import sys

import numpy as np
import pytest
import torch

import harness
import plain_litizen as plain
from litizen_models import MODELS, make_model

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
REPO = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = ["float32", "bfloat16"]
TD = {"float32": torch.float32, "bfloat16": torch.bfloat16}
TOL = {"float32": 2e-5, "bfloat16": 2e-2}


@pytest.fixture(scope="module")
def dirs(tmp_path_factory):
    root = tmp_path_factory.mktemp("litizen")
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


def _close(got, want, tol):
    assert (got.cpu().double() - want).abs().max() < tol * want.abs().max()


# ---- norms in groups ---------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,H,groups", [(3, 50, 5), (7, 96, 3), (300, 100, 25), (5, 1100, 11), (300, 1536, 4), (4, 4096, 256), (3, 6144, 2),
                                        (2, 9000, 9), (270, 4100, 5), (2, 20000, 8), (5, 384, 1)])
def test_norms_in_groups_of_the_stream_and_of_what_it_gets(T, H, groups, dtype):
    """A branch normed in groups (rows, and a stack of partial sums) beside plain ones and one normed over the row, and norms in
    groups of the new row, of all rows and of some; parts whose sizes differ by orders of magnitude."""
    from xinfer_amd import kernels
    dt = TD[dtype]
    g = torch.Generator().manual_seed(T + H)
    r = lambda *s: torch.randn(*s, generator=g)
    sizes = torch.repeat_interleave(10.0 ** torch.linspace(-1, 2, groups), H // groups)
    x, y, stack, low = r(T, H) * sizes, (r(T, H) * sizes.flip(0)).to(dt), r(3, T, H) * sizes.flip(0), r(T, H).to(dt)
    w1, w2, v = (1 + 0.2 * r(H) for _ in range(3))
    d = lambda t: t.to(DEV)
    tol = 5e-6 if dtype == "float32" else 8e-3
    for terms, norm_groups in (((), groups), (((y, w1, 1e-5, 1.0, groups),), groups),
                               (((stack, w2, 1e-3, 0.5, groups), (low, None, 0.0, 2.0)), groups),
                               (((y, w1, 1e-5, 1.0, groups), (stack, w2, 1e-4, -1.0)), 1), (((y, w1, 1e-5, 1.0),), groups)):
        s = x.double()
        for a, w, eps, f, *n in terms:
            b = a.double() if a.dim() == 2 else a.double().sum(0)
            s = s + f * (b if w is None else plain.group_norm(b, eps, w.double(), n[0] if n else 1))
        want = plain.group_norm(s, 1e-5, v.double(), norm_groups)
        dev = [(d(t[0]), None if t[1] is None else d(t[1]), *t[2:]) for t in terms]
        res, rounded, _, (h,) = kernels.stream_join(d(x), dev, [(d(v), 1e-5, norm_groups)], dt, keep=True, rounded=True)
        _close(res, s, 5e-6)
        _close(rounded, s, tol)
        _close(h, want, tol)
        rows = [T - 1, 0, T // 2]
        _close(kernels.stream_join(d(x), dev, [(d(v), 1e-5, norm_groups)], dt, rows=_i32(rows))[3][0], want[rows], tol)
    with pytest.raises(kernels.KernelError):
        kernels.stream_join(d(x), [(d(y), d(w1), 1e-5, 1.0, H + 1)], keep=True)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_grouped_norm_inside_other_arrangements(dtype):
    """What blocks that know nothing of open streams ask of a norm: before a sublayer, on some rows, on a branch's output."""
    from xinfer_amd.config.spec import PartSpec
    from xinfer_amd.parts import norm_class
    dt = TD[dtype]
    g = torch.Generator().manual_seed(3)
    part = norm_class("rmsnorm")(PartSpec("rmsnorm", dict(dim=60, eps=1e-5, groups=4, name="n")), dt)
    w = 1 + 0.2 * torch.randn(60, generator=g)
    part.weight = w.to(DEV)
    x, y = torch.randn(9, 60, generator=g), torch.randn(9, 60, generator=g).to(dt)
    tol = 5e-6 if dtype == "float32" else 8e-3
    resid = x.to(DEV)
    h = part.forward(resid, y.to(DEV), dt, add_scale=0.5)
    s = x.double() + 0.5 * y.double()
    _close(h, plain.group_norm(s, 1e-5, w.double(), 4), tol)
    _close(resid, s, 5e-6)
    some = part.forward(resid, None, dt, rows=_i32([7, 2]))
    _close(some, plain.group_norm(s, 1e-5, w.double(), 4)[[7, 2]], tol)
    low = part.forward_branch(resid, y.to(DEV), dt)
    s = s + plain.group_norm(y.double(), 1e-5, w.double(), 4)
    _close(resid, s, 5e-6)
    _close(low, s, tol)


# ---- a convolution in front of a mixer -------------------------------------------------------------------------------------
class _Ctx:
    """What the convolution reads of a step."""

    def __init__(self, slots, lens):
        cu = [0]
        for n in lens:
            cu.append(cu[-1] + n)
        self.num_tokens, self.num_seqs, self.max_q_len = cu[-1], len(lens), max(lens)
        self.state_slots, self.cu_q = _i64(slots), _i32(cu)
        self.tok_seq = _i32([b for b, n in enumerate(lens) for _ in range(n)])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("C,taps", [(50, 6), (96, 3), (64, 1), (260, 4), (33, 2), (1032, 5), (4096, 4)])
def test_short_convolutions_of_unequal_requests_in_portions(C, taps, dtype):
    """Three requests in slots that are not in order and were used before, in portions shorter than the taps, single tokens
    together (results and tails in one launch) and beside portions; with silu and a bias (in front of a state space) and as an
    addition to the input (in front of a mixer)."""
    from xinfer_amd.parts.short_conv import short_conv
    dt = TD[dtype]
    lens, cuts, slots = [40, 9, 25], [[2, 30, 1, 1, 1, 5], [1, 2, 1, 1, 1, 3], [7, 14, 1, 1, 1, 1]], [3, 0, 2]
    g = torch.Generator().manual_seed(C)
    u = [torch.randn(n, C, generator=g).to(dt) for n in lens]
    w, b, ib = torch.randn(C, taps, generator=g), torch.randn(C, generator=g), torch.randn(C, generator=g)
    for act, in_bias in (("silu", None), ("none", None), ("none", ib), ("silu", ib)):
        want = []
        for x in u:
            y = plain.causal_conv(x.double() + (0 if in_bias is None else in_bias.double()), w.double()) + b.double()
            want.append(plain.silu(y) if act == "silu" else y)
        tails = torch.full((5, taps - 1, C), 7.0, device=DEV) if taps > 1 else None
        if tails is not None:
            tails[slots] = 0
        got, at = [[] for _ in u], [0, 0, 0]
        for step in range(6):
            lens_now = [c[step] for c in cuts]
            # the convolution's channels lie in a longer packed row
            rows = torch.cat([torch.cat([x[at[i]:at[i] + n], x[at[i]:at[i] + n, :4]], dim=1) for i, (x, n) in enumerate(zip(u, lens_now))])
            y = short_conv(rows.to(DEV)[:, :C], w.to(DEV), b.to(DEV), tails, _Ctx(slots, lens_now), act=act,
                           in_bias=None if in_bias is None else in_bias.to(DEV)).cpu()
            k = 0
            for i, n in enumerate(lens_now):
                got[i].append(y[k:k + n])
                k += n
                at[i] += n
        for i in range(3):
            _close(torch.cat(got[i]), want[i], 2e-6 if dtype == "float32" else 6e-3)
            if taps > 1:
                last = u[i][-(taps - 1):].double() + (0 if in_bias is None else in_bias.double())
                assert (tails[slots[i]].cpu().double()[-last.shape[0]:] - last).abs().max() < 1e-6 * last.abs().max()
        if taps > 1:
            assert float((tails[[1, 4]] - 7.0).abs().max()) == 0                 # other requests' slots are left alone


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_mixer_behind_its_convolution(dtype):
    from xinfer_amd.config.spec import PartSpec
    from xinfer_amd.parts import LayerCache, Mixer, StateNeed, mixer_class, register_mixer

    @register_mixer("test_echo")
    class Echo(Mixer):
        graph_safe = True

        def state_need(self):
            return StateNeed((3,), torch.float32)

        def forward(self, x, ctx, cache):
            assert cache.state.shape[1:] == (3,)                              # the inner mixer finds its own state first
            return x

    dt, C, taps = TD[dtype], 48, 4
    part = mixer_class("input_conv")(PartSpec("input_conv", dict(hidden_size=C, taps=taps, name="c", inner=PartSpec("test_echo"))), dt)
    g = torch.Generator().manual_seed(1)
    w = (torch.randn(C, taps, generator=g) * 0.5).to(torch.bfloat16)

    class Store:
        def get(self, name, dtype=None, device="cpu"):
            return w.to(device=device, dtype=dtype)
    part.load(Store(), "p", DEV)
    assert part.graph_safe and [(n.name, n.shape) for n in part.state_need()] == [("state", (3,)), ("input_tail", (3, C))]
    h = torch.randn(30, C, generator=g).to(dt)
    states = {"state": torch.zeros(2, 3, device=DEV), "input_tail": torch.zeros(2, 3, C, device=DEV)}
    cache, out, at = LayerCache(state=states["state"], states=states), [], 0
    for n in (2, 1, 1, 17, 1, 8):
        out.append(part.forward(h[at:at + n].to(DEV), _Ctx([1], [n]), cache).cpu())
        at += n
    _close(torch.cat(out), plain.input_conv(h.double(), w.double()), 2e-6 if dtype == "float32" else 6e-3)
    frozen = states["input_tail"].clone()                    # a run that reads another run's cache moves nothing on
    for n in (1, 4):
        part.forward(h[:n].to(DEV), _Ctx([1], [n]), LayerCache(state=states["state"], states=states, write=False))
        assert torch.equal(states["input_tail"], frozen)


# ---- heads ------------------------------------------------------------------------------------------------------------------
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


def _turn_pairs(x, ang):
    """Neighbours (2i, 2i + 1) turned, for the option this family does not use."""
    c, s = ang.cos()[:, None, :], ang.sin()[:, None, :]
    out = x.clone()
    n = 2 * ang.shape[1]
    out[..., 0:n:2], out[..., 1:n:2] = x[..., 0:n:2] * c - x[..., 1:n:2] * s, x[..., 1:n:2] * c + x[..., 0:n:2] * s
    return out


HEAD_CASES = [  # H, G, d, dv, rot, page, keys are the values, norms, values turn, neighbours
    (6, 2, 16, 16, 10, 16, True, True, False, False), (4, 4, 128, 128, 128, 64, True, True, False, False),
    (3, 1, 12, 12, 6, 8, True, True, False, False), (2, 2, 96, 96, 96, 64, True, True, False, False),
    (5, 5, 20, 20, 0, 8, True, False, False, False), (6, 2, 16, 24, 8, 16, False, False, True, False),
    (4, 2, 64, 96, 32, 64, False, False, True, False), (3, 3, 128, 64, 64, 16, False, True, True, False),
    (3, 1, 20, 10, 4, 8, False, False, True, False), (2, 1, 8, 40, 0, 8, False, False, True, False),
    (2, 2, 16, 32, 16, 16, False, True, True, True), (4, 1, 64, 64, 48, 32, True, True, True, False),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("L", [45, 301])
@pytest.mark.parametrize("case", HEAD_CASES)
def test_heads_whose_values_are_the_keys_or_turn(case, L, dtype):
    """From a row that is longer than its heads (a gate behind them): norm, rotation, values from the keys as projected or turned
    by their own position, and the cache write, a head a wave and (many tokens, sizes in eights) eight dims a lane."""
    from xinfer_amd import kernels
    H, G, d, dv, rot, page, keyed, norms, turned, pairs = case
    dt, eps, grouped = TD[dtype], 1e-5, dtype == "bfloat16"
    g = torch.Generator().manual_seed(H * 10 + d)
    heads = (H + G) * d + (0 if keyed else G * dv)
    packed = torch.randn(L, heads + H * dv, generator=g).to(dt)
    qw, kw = (1 + 0.3 * torch.randn(d, generator=g), 1 + 0.3 * torch.randn(d, generator=g)) if norms else (None, None)
    full = packed.double()
    q, k = full[:, :H * d].view(L, H, d), full[:, H * d:(H + G) * d].view(L, G, d)
    v = k if keyed else full[:, (H + G) * d:heads].view(L, G, dv)
    if norms:
        q, k = plain.group_norm(q, eps, qw.double()), plain.group_norm(k, eps, kw.double())
    pos = torch.arange(L) + 700
    turn = _turn_pairs if pairs else plain.turn_halves
    kwargs = {}
    table_of = lambda a: torch.cat([torch.zeros(700, a.shape[1], dtype=a.dtype), a])         # the tables start at position 0
    if rot:
        a = plain.angles(90.0, rot, pos)
        q, k = turn(q, a), turn(k, a)
        kwargs = dict(cos=table_of(a.cos()).float().to(DEV), sin=table_of(a.sin()).float().to(DEV), rotary_dim=rot)
    if turned:
        a = plain.angles(90.0, dv, pos)
        v = turn(v, a)
        kwargs.update(v_cos=table_of(a.cos()).float().to(DEV), v_sin=table_of(a.sin()).float().to(DEV))
    k_pool, v_pool, table, slots = _pools(L, G, d, dv, page, dt, grouped, seed=d)
    k_pool, v_pool = k_pool.to(DEV), v_pool.to(DEV)
    slots[5] = -1                                                             # a token that stores nothing
    got = kernels.head_rows(packed.to(DEV)[:, :heads], slots.to(DEV), k_pool, v_pool, H, G, d, dv, v_grouped=grouped,
                            positions=pos.int().to(DEV), eps=eps, interleaved=pairs, values_in_keys=keyed,
                            q_weight=None if qw is None else qw.to(DEV), k_weight=None if kw is None else kw.to(DEV), **kwargs)
    tol = 1e-5 if dtype == "float32" else 6e-3
    _close(got, q, tol)
    gk, gv = _read_pools(k_pool.cpu(), v_pool.cpu(), table, L, grouped)
    keep = [p for p in range(L) if p != 5]
    _close(gk[keep], k[keep], tol)
    _close(gv[keep], v[keep], tol)
    assert float(gk[5].abs().max()) == 0 and float(gv[5].abs().max()) == 0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,H,dv", [(1, 6, 24), (3, 4, 96), (200, 3, 128), (9, 2, 10), (260, 5, 64), (4, 1, 18), (7, 3, 15)])
def test_results_turned_back_and_gated(T, H, dv, dtype):
    from xinfer_amd import kernels
    dt = TD[dtype]
    g = torch.Generator().manual_seed(T)
    x, packed = torch.randn(T, H * dv, generator=g).to(dt), torch.randn(T, 16 + H * dv, generator=g).to(dt) * 3
    pos = torch.randint(0, 3000, (T,), generator=g)
    tol = 2e-6 if dtype == "float32" else 8e-3
    gate, factor = packed.to(DEV)[:, 16:], torch.sigmoid(packed[:, 16:].double())
    _close(kernels.head_finish_(x.to(DEV), H, gate=gate), x.double() * factor, tol)
    if dv % 2:
        return
    full = plain.angles(77.0, dv, torch.arange(3000))
    kw = dict(cos=full.cos().float().to(DEV), sin=full.sin().float().to(DEV), positions=pos.int().to(DEV))
    for pairs, turn in ((False, plain.turn_halves), (True, _turn_pairs)):
        want = turn(x.double().view(T, H, dv), -full[pos]).reshape(T, H * dv)
        _close(kernels.head_finish_(x.to(DEV), H, interleaved=pairs, **kw), want, tol)
        _close(kernels.head_finish_(x.to(DEV), H, gate=gate, interleaved=pairs, **kw), want * factor, tol)


# ---- attention with sinks, in windows and chunks ------------------------------------------------------------------------------
def _planted(L, H, G, d, window, chunk, scale, height, seed):
    """q [L, H, d] and k [L, G, d] in which chosen (query, key) pairs have a score that stands out: keys just inside and just outside
    a window or chunk, at page borders, at the first tokens, far back."""
    g = torch.Generator().manual_seed(seed)
    q = torch.randn(L, H, d, generator=g) * 0.3
    k = torch.randn(L, G, d, generator=g) * 0.3
    big = height / scale
    c = chunk or window or L
    queries = set(range(max(0, L - 12), L)) | {1, 2, 17, 31, 32, 63, 64, 65, 128} | {e + o for e in range(0, L, c) for o in (-1, 0, 1, 2)}
    pairs = []
    for i in sorted(queries):
        if not (0 <= i < L):
            continue
        edge = i - i % c if chunk else i - c + 1
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


SEEN_CASES = [  # H, G, d, dv, window, chunk, cap, scale, L, page
    (6, 2, 16, 24, 0, 21, 9.0, 0.4, 90, 16),
    (6, 2, 16, 16, 19, 0, 0.0, 0.6, 90, 16),
    (5, 5, 20, 20, 1, 0, 0.0, 0.5, 40, 8),
    (3, 1, 12, 12, 3, 0, 0.0, 0.7, 61, 8),
    (3, 1, 20, 10, 0, 5, 6.0, 0.5, 61, 8),
    (2, 2, 8, 16, 0, 1, 8.0, 0.6, 40, 8),
    (4, 4, 128, 128, 100, 0, 0.0, 0.09, 330, 64),
    (2, 2, 96, 96, 70, 0, 0.0, 0.12, 260, 64),
    (6, 2, 64, 96, 0, 150, 15.0, 0.12, 400, 64),
    (8, 1, 64, 64, 0, 70, 10.0, 0.13, 300, 64),       # single tokens: the heads are the rows of a block
    (8, 1, 64, 64, 1000, 0, 0.0, 0.2, 260, 64),       # a window wider than the request
    (8, 1, 64, 64, 65, 0, 0.0, 0.15, 260, 64),
    (4, 2, 32, 32, 0, 0, 0.0, 0.3, 150, 16),          # everything is seen
    (4, 1, 64, 128, 0, 64, 7.0, 0.2, 200, 64),        # chunks as long as a page
]


def _seen_case(case, dtype, matrix_cores, tail, sink_kind):
    from xinfer_amd import kernels
    H, G, d, dv, window, chunk, cap, scale, L, page = case
    dt, grouped = TD[dtype], dtype == "bfloat16"
    height = 6.0 if cap == 0 else 0.8 * cap
    q, k = _planted(L, H, G, d, window, chunk, scale, height, seed=L)
    g = torch.Generator().manual_seed(L)
    v = torch.randn(L, G, dv, generator=g)
    q, k, v = q.to(dt), k.to(dt), v.to(dt)
    # a sink whose score is 0, or learned ones from below every score to above the planted ones
    sinks = torch.zeros(H) if sink_kind == "one" else torch.linspace(-12.0, height + 1.0, H)
    ref = lambda win, chk, snk: plain.softmax_heads(q.double(), k.double(), v.double(), scale,
                                                    plain.chunk_seen(L, chk) if chk else plain.window_seen(L, win), snk.double(), cap).reshape(L, H * dv)
    want = ref(window, chunk, sinks)
    others = [(window, chunk, sinks - 50.0)]                            # no sinks, and edges that are one off, would show
    if 0 < window < L:
        others += [(w, 0, sinks) for w in (window + 1, window - 1) if w > 0]
    if 0 < chunk < L:
        others += [(0, c, sinks) for c in (chunk + 1, chunk - 1) if c > 0]
    for o in others:
        assert (ref(*o) - want).abs().max() > 0.05 * want.abs().max()
    k_pool, v_pool, table, slots = _pools(L, G, d, dv, page, dt, grouped, seed=L)
    for p in range(L):
        pg, off = int(slots[p]) // page, int(slots[p]) % page
        k_pool[pg, :, off] = k[p]
        if grouped:
            v_pool[pg, :, off // 8, :, off % 8] = v[p]
        else:
            v_pool[pg, :, off] = v[p]
    k_pool, v_pool, table, sinks = k_pool.to(DEV), v_pool.to(DEV), table.to(DEV), sinks.to(DEV)

    class Ctx:
        pass

    def run(positions):
        qs, pos = q[positions[0]:positions[-1] + 1].to(DEV), _i32(positions)
        if not matrix_cores:
            return kernels.attention_generic(qs, k_pool, v_pool, table, torch.zeros_like(pos), pos, scale, window, v_grouped=grouped,
                                             softcap=cap, chunk=chunk, sinks=sinks)
        # through the engine's chooser: portions, single tokens in slices, heads as the rows of a block
        n, ctx = len(positions), Ctx()
        ctx.block_tables, ctx.tok_seq, ctx.positions, ctx.scratch = [table], torch.zeros_like(pos), pos, {}
        ctx.num_seqs, ctx.max_q_len, ctx.max_ctx_len = 1, n, positions[-1] + 1
        ctx.cu_q, ctx.ctx_lens, ctx.cu_q_host, ctx.ctx_lens_host = _i32([0, n]), _i32([positions[-1] + 1]), [0, n], [positions[-1] + 1]
        return kernels.attention(qs, k_pool, v_pool, ctx, 0, scale, window, v_grouped=grouped, softcap=cap, sinks=sinks, chunk=chunk)
    head = max(1, L - tail)
    cuts = [0, head // 3 + 1, head] if head > 8 else [0, head]
    outs = [run(list(range(a, b))) for a, b in zip(cuts[:-1], cuts[1:]) if b > a] + [run([p]) for p in range(head, L)]
    got = torch.cat([o.cpu() for o in outs]).double()
    err = (got - want).abs().max(dim=1).values
    bad = (err > TOL[dtype] * want.abs().max()).nonzero()
    assert bad.numel() == 0, f"first wrong position {int(bad[0])} of {L}: {float(err[int(bad[0])]):.3e}"


@pytest.mark.parametrize("sink_kind", ["one", "learned"])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", SEEN_CASES)
def test_attention_with_sinks_and_planted_keys(case, dtype, sink_kind):
    _seen_case(case, dtype, matrix_cores=False, tail=9, sink_kind=sink_kind)


@pytest.mark.parametrize("sink_kind", ["one", "learned"])
@pytest.mark.parametrize("case", [c for c in SEEN_CASES if c[2] % 8 == 0 and c[3] % 8 == 0])
def test_attention_with_sinks_on_the_matrix_cores(case, sink_kind):
    _seen_case(case, "bfloat16", matrix_cores=True, tail=9, sink_kind=sink_kind)
    _seen_case(case, "bfloat16", matrix_cores=True, tail=75, sink_kind=sink_kind)


# ---- experts -----------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,I,top,T,H", [(4, 1, 2, 5, 96), (5, 3, 8, 40, 50), (8, 3, 3, 300, 384), (200, 56, 10, 7, 128), (3, 0, 1, 9, 64),
                                         (1, 1, 1, 6, 40)])
def test_choice_by_corrected_scores(E, I, top, T, H, dtype):
    from xinfer_amd import kernels
    A = E + I
    g = torch.Generator().manual_seed(E)
    x, r, c = torch.randn(T, H, generator=g).to(TD[dtype]), torch.randn(A, H, generator=g) / H ** 0.5 * 2, torch.randn(A, generator=g) * 0.2
    chosen, wt = plain.route(x.double(), r.double(), c.double(), top)
    key = (torch.softmax(x.double() @ r.double().T, -1) + c.double()).sort(-1, descending=True).values
    idx, w = kernels.moe_route(x.to(DEV), r.to(DEV), None, top, all_scores=True, correction=c.to(DEV))
    clear = torch.ones(T, dtype=torch.bool) if top == A else (key[:, top - 1] - key[:, top]) > 1e-5
    order = (key[:, :top - 1] - key[:, 1:top]).min(dim=-1).values > 1e-5 if top > 1 else clear
    keep = clear & order
    assert int(keep.sum()) > 0.8 * T
    assert torch.equal(idx.cpu().long()[keep], chosen[keep])
    assert (w.cpu().double()[keep] - wt[keep]).abs().max() < 2e-6
    # sigmoids, chosen with the correction and taken as they are
    s = torch.sigmoid(x.double() @ r.double().T)
    idx, w = kernels.moe_route(x.to(DEV), r.to(DEV), None, top, sigmoid=True, correction=c.to(DEV))
    best = (s + c.double()).sort(-1, descending=True)
    keep = (best.values[:, :-1] - best.values[:, 1:])[:, :top].min(dim=-1).values > 1e-5 if A > 1 and top < A else torch.zeros(T, dtype=torch.bool)
    assert torch.equal(idx.cpu().long()[keep], best.indices[keep][:, :top])
    if bool(keep.any()):
        assert (w.cpu().double()[keep] - torch.gather(s, 1, best.indices[:, :top])[keep]).abs().max() < 2e-6
    with pytest.raises(kernels.KernelError):
        kernels.moe_route(x.to(DEV), r.to(DEV), None, top, correction=c.to(DEV))


@pytest.mark.parametrize("form", ["pairs", "grouped", "library"])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,I,top,T,H,F", [(4, 2, 3, 5, 96, 48), (8, 3, 4, 150, 384, 64), (3, 1, 2, 300, 104, 40), (5, 2, 4, 33, 50, 22),
                                           (2, 2, 4, 40, 64, 32)])
def test_identity_experts_and_a_shared_branch(E, I, top, T, H, F, dtype, form):
    """A pair whose expert has no tensors gets its weight times the input; tokens that choose identity experts alone; a further
    row added where the experts' rows are summed; in every form of the experts' products."""
    from xinfer_amd import kernels
    dt = TD[dtype]
    if form != "pairs" and dtype == "float32":
        pytest.skip("the float32 path takes a pair at a time")
    if form == "grouped" and not kernels.moe_grouped_takes(T, top, E, H, F, dt, force=True):
        pytest.skip("sizes in eights only")
    g = torch.Generator().manual_seed(T)
    x, add = torch.randn(T, H, generator=g).to(dt), torch.randn(T, H, generator=g).to(dt)
    gu = (torch.randn(E, 2 * F, H, generator=g) / H ** 0.5).to(dt)
    dn = (torch.randn(E, H, F, generator=g) / F ** 0.5).to(dt)
    idx = torch.stack([torch.randperm(E + I, generator=g)[:top] for _ in range(T)])
    if I >= 2 and top <= I:
        idx[0, :] = torch.arange(E, E + top)
    wt = torch.rand(T, top, generator=g)
    want = torch.zeros(T, H, dtype=torch.float64)
    for t in range(T):
        for e, c in zip(idx[t].tolist(), wt[t].double()):
            w = {"gate": gu[e, :F].double(), "up": gu[e, F:].double(), "down": dn[e].double()} if e < E else None
            want[t] += c * (x[t].double() if e >= E else plain.gated(x[t].double(), w))
    args = [t.to(DEV) for t in (x, gu, dn, idx.int(), wt)]
    run = (lambda **kw: kernels.moe_experts_library(*args, identity=I, **kw)) if form == "library" else (
        lambda **kw: kernels.moe_experts(*args, grouped=form == "grouped", identity=I, **kw))
    tol = 5e-6 if dtype == "float32" else 1e-2
    _close(run(), want, tol)
    _close(run(add=add.to(DEV)), want + add.double(), tol)


# ---- whole models ----------------------------------------------------------------------------------------------------
LENGTHS = {"A": [1, 2, 19, 22, 43, 77, 130], "B": [3, 8, 9, 18, 64, 101], "C": [1, 5, 6, 40, 75, 210], "M": [2, 1, 30, 140],
           "R": [5, 101, 330, 64, 301], "S": [3, 70, 71, 260, 129]}


def _requests(name):
    rng = random.Random(900 + ord(name))
    vocab = MODELS[name]["config"]["vocab"]
    return {f"r{i}": harness.random_prompt(rng, n, vocab) for i, n in enumerate(LENGTHS[name])}


_plain_cache = {}
_model_cache = {}


def _plain_logits(name, model_dir):
    if name not in _plain_cache:
        pm = plain.PlainLitizen(model_dir, torch.float64)
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


def test_the_routers_choices_are_clear_and_vary(dirs):
    for name in MODELS:
        pm = plain.PlainLitizen(dirs(name), torch.float64)
        for toks in _requests(name).values():
            for i, l in enumerate(pm.cfg["layers"]):
                ml = l.get("mlp")
                if not ml or ml["kind"] != "moe" or len(toks) < 60:
                    continue
                x = pm.stream(toks)[i]
                h = plain.input_conv(pm.norm(x, f"l{i}.norm1"), pm.w[f"l{i}.canon1"])
                h = pm.norm(x + pm.norm(pm.mixer(i, h, torch.arange(len(toks))), f"l{i}.norm1b"), f"l{i}.norm2")
                w = plain.sub(pm.w, f"l{i}.mlp.")
                s = (torch.softmax(h @ w["router"].T, -1) + w["correction"]).sort(-1, descending=True)
                top, n = ml["router"]["top"], w["router"].shape[0]
                assert top == n or float((s.values[:, top - 1] - s.values[:, top]).min()) > 0.015
                if ml["router"].get("identity"):
                    assert bool((s.indices[:, :top] >= ml["router"]["experts"]).any())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MODELS))
def test_whole(name, dtype, dirs):
    got, _ = _run(name, dtype, dirs, harness.trace_whole(_requests(name)), "whole")
    assert len(got) == sum(LENGTHS[name])


@pytest.mark.parametrize("name", list(MODELS))
def test_the_stream_after_every_layer(name, dirs):
    """float32, one request: the stream after every layer against the plain one."""
    from xinfer_amd.engine import ModelRunner, StepEntry
    from xinfer_amd.parts.joining import join
    model = _model(name, "float32", dirs(name))
    toks = _requests(name)["r3"]
    want = plain.PlainLitizen(dirs(name), torch.float64).stream(toks)[1:]
    seen, kept = [], [(b, b.forward) for b in model.blocks]
    try:
        for b, orig in kept:
            def fwd(stream, ctx, cache, _o=orig):
                s = _o(stream, ctx, cache)
                assert s.open                                                   # a layer leaves its last branch to the next pass
                seen.append(join(s, torch.float32)[0].resid.cpu().double())
                return s
            b.forward = fwd
        runner = ModelRunner(model, page_size=MODELS[name]["page_size"], num_pages=20, max_requests=1, use_graphs=False)
        runner.add_request(0)
        runner.step([StepEntry(0, toks, [])])
    finally:
        for b, _ in kept:
            del b.forward
    assert len(seen) == len(want)
    for i, (a, b) in enumerate(zip(seen, want)):
        assert (a - b).abs().max() < 2e-5 * b.abs().max(), f"layer {i}"


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_sandwich_of_norms_that_the_pass_cannot_make(dtype, dirs):
    """The same layers with their norms run one by one on a joined stream, and a pre-norm layer in between."""
    from dataclasses import replace
    from xinfer_amd.engine import ModelRunner, StepEntry
    from xinfer_amd.engine.model import CausalLM
    from xinfer_amd.models import config_from_dict
    from xinfer_amd.weights.store import SafetensorsStore
    fam, cfg = config_from_dict(MODELS["A"]["config"])
    spec = fam.spec(cfg)
    layers = list(spec.layers)
    norms = layers[1].norms
    layers[1] = replace(layers[1], block="prenorm", norms={k: norms[k] for k in ("norm1", "norm2")})
    model = CausalLM(replace(spec, layers=tuple(layers)), TD[dtype]).load(SafetensorsStore(dirs("A")), DEV)
    model.blocks[0].joined = model.blocks[2].joined = False
    assert model.blocks[0].writes_stream and not model.blocks[3].writes_stream
    runner = ModelRunner(model, page_size=16, num_pages=12, max_requests=1, use_graphs=False)
    runner.add_request(0)
    toks = _requests("A")["r5"]
    got = torch.cat([runner.step([StepEntry(0, toks[a:b], list(range(b - a)))]).cpu() for a, b in ((0, 30), (30, 31), (31, len(toks)))])

    class Mixed(plain.PlainLitizen):
        def norm(self, x, name):
            return x if name in ("l1.norm1b", "l1.norm2b") else super().norm(x, name)
    want = Mixed(dirs("A"), torch.float64).logits(toks)
    assert (got.double() - want).abs().max() < harness.TOL[dtype] * want.abs().max()


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
    """More requests than state slots, one after the other in the same slots and pages: a request that starts finds no
    state and no inputs of the one before."""
    for seed in (1, 2):
        _run(name, dtype, dirs, harness.trace_mixed(_requests(name), seed, max_live=3), f"mixed {seed}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "R", "M"])
def test_short_chunks_of_the_states_walks(name, dtype, dirs, monkeypatch):
    from xinfer_amd import kernels
    monkeypatch.setattr(kernels, "SCAN_CHUNK", 16)
    _run(name, dtype, dirs, harness.trace_whole(_requests(name)), "whole, chunks of 16")
    _run(name, dtype, dirs, harness.trace_portions(_requests(name), sizes=(33, 2, 47, 32, 5)), "portions, chunks of 16")
    _run(name, dtype, dirs, harness.trace_mixed(_requests(name), 3, max_live=3, sizes=(40, 2, 35, 64)), "mixed, chunks of 16")


@pytest.mark.parametrize("name", ["R", "S"])
def test_every_form_of_the_experts_products(name, dirs, monkeypatch):
    from xinfer_amd import kernels
    steps = harness.trace_mixed(_requests(name), 5, max_live=3, sizes=(40, 2, 35, 64))
    monkeypatch.setattr(kernels, "MOE_LIBRARY_ROWS", 1)
    _run(name, "bfloat16", dirs, steps, "library products")
    monkeypatch.setattr(kernels, "MOE_LIBRARY_ROWS", 1 << 20)
    _run(name, "bfloat16", dirs, steps, "grouped products")
    monkeypatch.setattr(kernels, "MOE_GROUPED", False)
    _run(name, "bfloat16", dirs, steps, "a pair at a time")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B", "C", "R", "S"])
def test_unequal_requests_decoding_together(name, dtype, dirs):
    reqs = {k: v for k, v in _requests(name).items() if len(v) > 8}
    reqs = dict(list(reqs.items())[:4])
    _run(name, dtype, dirs, harness.trace_batch_decode(reqs, tail=7), "batch decode", use_graphs=False)
    got, runner = _run(name, dtype, dirs, harness.trace_batch_decode(reqs, tail=7), "batch decode, graphs", graph_after=1)
    assert runner.graph_replays > 0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "R"])
def test_long_decoding(name, dtype, dirs):
    """Three tokens of prompt, then the rest one by one: states and inputs move on token by token, windows pass and chunks end under
    decoding, over several pages."""
    from xinfer_amd.engine import ModelRunner
    n = 253 if name == "A" else 340
    toks = harness.random_prompt(random.Random(9), n, MODELS[name]["config"]["vocab"])
    ref = {"a": plain.PlainLitizen(dirs(name), torch.float64).logits(toks).float()}
    steps = harness.trace_tail_one_by_one({"a": toks}, tail=n - 3)
    page = MODELS[name]["page_size"]
    runner = ModelRunner(_model(name, dtype, dirs(name)), page_size=page, num_pages=-(-n // page) + 1, max_requests=2, graph_after=2)
    got = harness.replay(runner, steps)
    assert runner.graph_replays > 200
    harness.compare(got, ref, harness.TOL[dtype], f"long decoding {name} {dtype}")


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
def test_greedy_generation_through_the_engine(dtype, dirs):
    """The framework's own entry point and scheduler: five prompts, three at a time, prompts cut into portions of 16
    tokens, greedy tokens against the plain implementation."""
    from xinfer_amd import Engine, EngineConfig, SamplingParams
    name = "A"
    rng = random.Random(3)
    vocab = MODELS[name]["config"]["vocab"]
    prompts = [harness.random_prompt(rng, n, vocab) for n in (5, 40, 17, 33, 2)]
    eng = Engine(EngineConfig(weight_path=dirs(name), page_size=16, num_pages=24, max_num_seqs=3, prefill_chunk_size=16,
                              max_model_len=128, seed=1), dtype)
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=24, ignore_eos=True))
    pm = plain.PlainLitizen(dirs(name), torch.float64)
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
    pm = plain.PlainLitizen(dirs(name), torch.float64)
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
    """float32: steps replayed from a recorded graph give the bits of the same steps launched one by one (states and inputs
    are advanced once a step, in the step that records too)."""
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
