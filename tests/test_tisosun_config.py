"""Tisosun's configuration, its turning into a model description, and the plain implementation's own pins, on the CPU."""
import copy
import math

import pytest
import torch

import plain_tisosun as plain
from tisosun_models import MODELS
from xinfer_amd.config.model_config import ConfigError
from xinfer_amd.models import config_from_dict, family_of


def test_config_round_trip_and_registry():
    for name, t in MODELS.items():
        fam, cfg = config_from_dict(t["config"])
        assert fam is family_of("Tisosun") and cfg.architecture == "Tisosun"
        assert fam.config_class.from_dict(cfg.to_dict()) == cfg and cfg.to_dict() == t["config"]
        assert len(cfg.layers) == len(t["config"]["layers"])


def test_what_the_layers_keep_and_what_their_tensors_are_called():
    from xinfer_amd.engine.model import CausalLM
    fam, cfg = config_from_dict(MODELS["A"]["config"])
    spec = fam.spec(cfg)
    assert [(e.layer, [op.kind for op in e.after]) for e in spec.schedule] == [(i, ["token_side", "depth_average"]) for i in range(4)]
    names = {d.name: tuple(d.shape) for d in CausalLM.declare(spec)}
    for want, shape in (("embed", (311, 96)), ("embed.norm", (96,)), ("side.embed", (311, 48)), ("l0.mix.y", (120, 96)),
                        ("l0.mix.x.b", (120,)), ("l0.mix.conv", (120, 3)), ("l0.mix.ra", (3, 40, 40)), ("l0.mix.ri.b", (3, 40)),
                        ("l0.mix.lam", (120,)), ("l0.mix.o", (96, 120)), ("l1.mix.left.q", (96, 96)), ("l1.mix.left.k.b", (32,)),
                        ("l1.mix.left.v", (48, 96)), ("l1.mix.left.k.norm", (16,)), ("l1.mix.left.o", (96, 144)),
                        ("l1.mix.right.g", (60, 96)), ("l1.mix.right.norm", (60,)), ("l1.mix.left.out", (96,)),
                        ("l1.mix.right.out", (96,)), ("l2.mix.z.b", (72,)), ("l2.mix.g", (72, 96)), ("l3.dwa", (5,)), ("l0.dwa", (2,)),
                        ("l2.side.gate", (12, 96)), ("l2.side.proj", (96, 12)), ("l2.side.norm", (96,)), ("l3.mlp.down", (96, 96)),
                        ("final.norm", (96,)), ("head", (311, 96))):
        assert names.get(want) == shape, want
    assert not any(n.startswith(("l2.mlp", "l2.norm2", "l0.mix.conv.w", "l1.mix.out")) for n in names)
    model = CausalLM(spec, torch.float32)
    # a layer's chunks are a window of that many tokens to the cache; layers of one size share a group
    assert sorted(model.kv_needs) == [1, 3] and sorted(g.window for g in model.cache_groups) == [21, 34]
    assert sorted(model.state_needs) == [0, 1, 2, 3] and model.state_needs[1].shape == (3, 12, 20)
    state, tail = model.state_needs[0]
    assert state.shape == (120,) and tail.shape == (2, 120) and tail.name == "conv_tail" and model.state_needs[2].shape == (72,)
    left = model.blocks[1].mixer.branches[0][2]
    assert left.by_head and left.head_norm and left.chunk == 21 and left.softcap == 15.0 and left.position.interleaved and left.position.precise
    assert model.blocks[0].norms[0].weight_offset == 1.0 and model.final_norm.weight_offset == 1.0 and model.embedding.norm["offset"] == 1.0
    # nothing of the model changes the stream's tensor in place: the embedding's output needs no copy
    assert model._keep_first and not model._copy_first
    fam, cfg = config_from_dict(MODELS["M"]["config"])
    assert not CausalLM(fam.spec(cfg), torch.bfloat16).kv_needs
    fam, cfg = config_from_dict(MODELS["C"]["config"])
    spec = fam.spec(cfg)
    assert not any("side" in d.name for d in CausalLM.declare(spec)) and [op.kind for op in spec.schedule[1].after] == ["depth_average"]
    model = CausalLM(spec, torch.bfloat16)
    assert model.state_needs[2][1].shape == (5, 42) and model.blocks[2].ffn is None and len(model.blocks[2].norms) == 1


@pytest.mark.parametrize("change,message", [
    (lambda c: c["layers"][0].update(type="conv"), "unknown layer type"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=4), "kv heads"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=7), "even"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=18), "rotated dims"),
    (lambda c: c["layers"][1]["mixer"]["left"]["mask"].update(size=0), "mask.size"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(softcap=-1.0), "softcap"),
    (lambda c: c["layers"][1]["mixer"]["right"]["decay"].pop(), "decays"),
    (lambda c: c["layers"][0]["mixer"].update(blocks=7), "blocks"),
    (lambda c: c["layers"][0]["mixer"].update(conv=0), "taps"),
    (lambda c: c["layers"][2]["mixer"].pop("width"), "width"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "mlp kind"),
    (lambda c: c["token_side"].update(dim=0), "token_side"),
    (lambda c: c.pop("norm"), "norm"),
])
def test_configurations_that_cannot_be_run(change, message):
    raw = copy.deepcopy(MODELS["A"]["config"])
    change(raw)
    with pytest.raises(ConfigError, match=message):
        config_from_dict(raw)


def test_how_long_portions_are_cut():
    from xinfer_amd import kernels
    rows = kernels.channel_items([1, 100, 63, 64], 32)
    assert rows[0] == (0, 1, 0, 0, 1)
    assert rows[1:5] == [(1, 33, 1, 1, 4), (33, 65, 1, 1, 4), (65, 97, 1, 1, 4), (97, 101, 1, 1, 4)]
    assert rows[5] == (101, 164, 2, 5, 1) and rows[6:] == [(164, 196, 3, 6, 2), (196, 228, 3, 6, 2)]
    assert kernels.channel_chunk(10) == kernels.CHANNEL_CHUNK and kernels.channel_chunk(8192) % 8 == 0
    assert -(-8192 // kernels.channel_chunk(8192)) <= kernels.CHANNEL_CHUNKS


def test_a_table_that_layers_share_is_loaded_once():
    from xinfer_amd.weights.store import RandomStore, TensorDecl
    store = RandomStore([TensorDecl("t", (5, 8))], 1)
    assert store.shared("t", torch.float32, "cpu") is store.shared("t", torch.float32, "cpu")
    assert store.shared("t", torch.bfloat16, "cpu") is not store.shared("t", torch.float32, "cpu")
    assert torch.equal(store.shared("t", torch.float32, "cpu"), store.get("t", torch.float32, "cpu"))


# ---- tables of the rotation --------------------------------------------------------------------------------------
def test_tables_in_float64_rounded_once():
    from xinfer_amd.config.spec import PartSpec
    from xinfer_amd.parts import position_encoding_class
    rot = dict(dims=12, base=300.0, scaling=dict(factor=5.0, original=90, fast=6.0, slow=1.0))
    part = position_encoding_class("rope")(PartSpec("rope", dict(
        head_dim=16, rotary_dim=12, theta=300.0, max_positions=3000, interleaved=True, precise=True,
        scaling=dict(kind="ramp", factor=5.0, original=90, fast=6.0, slow=1.0))), torch.float32)
    part.load(None, "", "cpu")
    f, grow = plain.rotary_frequencies(rot)
    ang = torch.arange(3000, dtype=torch.float64)[:, None] * f
    assert torch.equal(part.cos, (ang.cos() * grow).float()) and torch.equal(part.sin, (ang.sin() * grow).float())
    assert grow == 0.1 * math.log(5.0) + 1.0 and float(f[0]) == 1.0 and abs(float(f[-1]) - 300.0 ** (-10 / 12) / 5.0) < 1e-12


# ---- what fixes each rule of the plain implementation beside its text ------------------------------------------------
def test_chunks_are_counted_from_the_first_position():
    seen = plain.chunk_seen(7, 3)
    want = [[0], [0, 1], [0, 1, 2], [3], [3, 4], [3, 4, 5], [6]]
    assert [row.nonzero().flatten().tolist() for row in seen] == want
    assert plain.chunk_seen(5, None).sum() == 15 and torch.equal(plain.chunk_seen(4, 1), torch.eye(4, dtype=torch.bool))


def test_rotation_turns_neighbours():
    x = torch.randn(5, 2, 12, dtype=torch.float64)
    rot = dict(dims=8, base=100.0)
    y = plain.rotate_pairs(x, rot, torch.arange(5))
    assert torch.equal(y[0], x[0]) and torch.equal(y[..., 8:], x[..., 8:])
    a = 3 * 100.0 ** (-2 / 8)       # position 3, pair 1: dims 2 and 3
    assert torch.allclose(y[3, 0, 2], x[3, 0, 2] * math.cos(a) - x[3, 0, 3] * math.sin(a))
    assert torch.allclose(y[3, 0, 3], x[3, 0, 3] * math.cos(a) + x[3, 0, 2] * math.sin(a))


def test_recurrences_go_on_where_a_portion_ended():
    g = torch.Generator().manual_seed(1)
    a = torch.rand(9, 4, generator=g, dtype=torch.float64)
    b = torch.randn(9, 4, generator=g, dtype=torch.float64)
    S, last = plain.channel_recurrence(a, b)
    S1, mid = plain.channel_recurrence(a[:5], b[:5])
    S2, end = plain.channel_recurrence(a[5:], b[5:], mid)
    assert torch.allclose(torch.cat([S1, S2]), S) and torch.allclose(end, last) and torch.allclose(S[0], b[0])
    q, k = (torch.randn(6, 2, 3, generator=g, dtype=torch.float64) for _ in range(2))
    v = torch.randn(6, 2, 5, generator=g, dtype=torch.float64)
    o, end = plain.decayed_state(q, k, v, [0.5, 1.0])
    o1, mid = plain.decayed_state(q[:2], k[:2], v[:2], [0.5, 1.0])
    o2, end2 = plain.decayed_state(q[2:], k[2:], v[2:], [0.5, 1.0], mid)
    assert torch.allclose(torch.cat([o1, o2]), o) and torch.allclose(end2, end)
    assert torch.allclose(o[1, 0], 0.5 * (q[1, 0] @ k[0, 0]) * v[0, 0] + (q[1, 0] @ k[1, 0]) * v[1, 0])


def test_gates_of_the_recurrences():
    z, u = torch.tensor([[0.0, 2.0]], dtype=torch.float64), torch.tensor([[-1.0, 3.0]], dtype=torch.float64)
    a, b = plain.mingru_terms(z, u)
    assert torch.allclose(a + torch.sigmoid(z), torch.ones_like(a))
    assert torch.allclose(b[0, 0], 0.5 * torch.sigmoid(u[0, 0])) and torch.allclose(b[0, 1], torch.sigmoid(z[0, 1]) * 3.5)
    lam = torch.tensor([-3.0, 1.0], dtype=torch.float64)
    a, b = plain.rglru_terms(u, z, z + 1, lam)
    want = torch.exp(-8 * torch.sigmoid(z) * torch.log(1 + torch.exp(lam)))
    assert torch.allclose(a, want) and torch.allclose(b, torch.sqrt(1 - want ** 2) * torch.sigmoid(z + 1) * u)
    w = torch.arange(8, dtype=torch.float64).view(2, 2, 2)
    x = torch.tensor([[1.0, 2.0, 3.0, 4.0]], dtype=torch.float64)
    assert plain.block_gate(x, w, torch.zeros(2, 2, dtype=torch.float64)).tolist() == [[2.0, 8.0, 4 * 3 + 5 * 4, 6 * 3 + 7 * 4]]


def test_the_convolution_sees_nothing_before_a_sequence():
    g = torch.Generator().manual_seed(2)
    u = torch.randn(6, 2, generator=g, dtype=torch.float64)
    w = torch.randn(2, 3, generator=g, dtype=torch.float64)
    b = torch.tensor([0.5, -1.0], dtype=torch.float64)
    out = plain.short_conv(u, w, b)
    assert torch.allclose(out[0], b + w[:, 2] * u[0]) and torch.allclose(out[2], b + w[:, 0] * u[0] + w[:, 1] * u[1] + w[:, 2] * u[2])


def test_what_goes_on_is_a_sum_over_the_depth():
    x = [torch.full((2, 3), float(v)) for v in (1, 10, 100)]
    assert float(plain.depth_average([0.5, 0.25, 2.0], x)[0, 0]) == 0.5 + 2.5 + 200.0
