"""Litizen's configuration, its turning into a model description, and the plain implementation's own pins, on the CPU."""
import copy
import math

import pytest
import torch

import plain_litizen as plain
from litizen_models import MODELS
from xinfer_amd.config.model_config import ConfigError
from xinfer_amd.models import config_from_dict, family_of


def test_config_round_trip_and_registry():
    for name, t in MODELS.items():
        fam, cfg = config_from_dict(t["config"])
        assert fam is family_of("Litizen") and cfg.architecture == "Litizen"
        assert fam.config_class.from_dict(cfg.to_dict()) == cfg and cfg.to_dict() == t["config"]
        assert len(cfg.layers) == len(t["config"]["layers"])


def test_what_the_layers_keep_and_what_their_tensors_are_called():
    from xinfer_amd.engine.model import CausalLM
    fam, cfg = config_from_dict(MODELS["A"]["config"])
    spec = fam.spec(cfg)
    assert [e.layer for e in spec.schedule] == [0, 1, 2, 3] and all(l.block == "sandwich" for l in spec.layers)
    names = {d.name: tuple(d.shape) for d in CausalLM.declare(spec)}
    for want, shape in (("embed", (311, 96)), ("l0.canon1", (96, 3)), ("l0.norm1", (96,)), ("l0.norm1b", (96,)), ("l2.norm2b", (96,)),
                        ("l0.mix.q", (96, 96)), ("l0.mix.k", (32, 96)), ("l0.mix.v", (48, 96)), ("l0.mix.g", (144, 96)),
                        ("l0.mix.o", (96, 144)), ("l0.mix.sink", (6,)), ("l0.mlp.router", (5, 96)), ("l0.mlp.correction", (5,)),
                        ("l0.mlp.e3.down", (96, 48)), ("l0.mlp.shared.gate", (40, 96)), ("l1.mix.in", (160 + 48 + 4, 96)),
                        ("l1.mix.conv", (128, 4)), ("l1.mix.dt_bias", (4,)), ("l1.mix.norm", (80,)), ("l1.mlp.down", (96, 128)),
                        ("l2.mix.q.norm", (16,)), ("l2.mix.k.norm", (16,)), ("l2.mix.g", (96, 96)), ("l2.mlp.router", (7, 96)),
                        ("l3.canon1", (96, 3)), ("final.norm", (96,)), ("head", (311, 96))):
        assert names.get(want) == shape, want
    assert not any(n.startswith(("l2.mix.v", "l2.mix.sink", "l0.mix.q.norm", "l3.mlp", "l3.norm2", "l2.mlp.shared", "l0.mlp.e4"))
                   for n in names)
    model = CausalLM(spec, torch.float32)
    # a layer's chunks are a window of that many tokens to the cache
    assert sorted(model.kv_needs) == [0, 2] and sorted(g.window for g in model.cache_groups) == [19, 21]
    keep = {i: {s.name: s.shape for s in need} for i, need in model.state_needs.items()}
    assert keep == {0: {"input_tail": (2, 96)}, 1: {"state": (4, 12, 20), "conv_tail": (3, 128), "input_tail": (2, 96)},
                    2: {"input_tail": (2, 96)}, 3: {"state": (3, 24, 16), "conv_tail": (1, 96), "input_tail": (2, 96)}}
    assert model.state_needs[1][0].name == "state"                      # the inner mixer's own comes first
    turned, keyed = model.blocks[0].mixer.inner, model.blocks[2].mixer.inner
    assert turned.chunk == 21 and turned.window == 0 and turned.softcap == 9.0 and turned.sink_kind == "learned" and turned.gate
    assert turned.value_position.rotary_dim == 24 and turned.position.rotary_dim == 8 and not turned.head_norm
    assert keyed.values_in_keys and keyed.window == 19 and keyed.chunk == 0 and keyed.sink_kind == "one" and keyed.head_norm
    assert not keyed.position.interleaved and keyed.position.precise and keyed.value_position is None
    assert model.blocks[0].norms[0].groups == 3 and model.final_norm.groups == 3 and not model.final_norm.foldable
    assert model.head.softcap == 12.0 and model.embedding.scale == 0.7 and model.graph_safe
    fam, cfg = config_from_dict(MODELS["M"]["config"])
    assert not CausalLM(fam.spec(cfg), torch.bfloat16).kv_needs
    fam, cfg = config_from_dict(MODELS["B"]["config"])
    model = CausalLM(fam.spec(cfg), torch.bfloat16)
    assert 0 not in model.state_needs and [s.name for s in model.state_needs[2]] == ["state"]      # one tap keeps nothing
    assert model.blocks[0].norms[0].foldable and model.blocks[1].ffn is None and len(model.blocks[1].norms) == 2


@pytest.mark.parametrize("change,message", [
    (lambda c: c["layers"][0].update(type="conv"), "unknown layer type"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), "kv heads"),
    (lambda c: c["layers"][2]["mixer"].update(vdim=24), "keys have the keys'"),
    (lambda c: c["layers"][0]["mixer"].update(vdim=23), "in pairs"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "even"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18), "at most"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "mask.size"),
    (lambda c: c["layers"][0]["mixer"].update(softcap=-1.0), "softcap"),
    (lambda c: c["layers"][1]["mixer"].update(groups=3), "groups"),
    (lambda c: c["layers"][1]["mixer"].pop("state"), "state"),
    (lambda c: c["layers"][0]["mlp"].update(kind="wide"), "mlp kind"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=6), "experts"),
    (lambda c: c["layers"][0]["mlp"]["shared"].update(ff=0), "shared"),
    (lambda c: c["norm"].update(groups=7), "norm.groups"),
    (lambda c: c["canon"].update(taps=0), "canon.taps"),
    (lambda c: c.update(logit_softcap=0.0), "logit_softcap"),
    (lambda c: c.pop("norm"), "norm"),
])
def test_configurations_that_cannot_be_run(change, message):
    raw = copy.deepcopy(MODELS["A"]["config"])
    change(raw)
    with pytest.raises(ConfigError, match=message):
        config_from_dict(raw)


def test_options_that_do_not_go_together():
    from xinfer_amd.config.spec import PartSpec
    from xinfer_amd.parts import mixer_class
    rope = lambda dims, head, inter=False: PartSpec("rope", dict(head_dim=head, rotary_dim=dims, theta=100.0, max_positions=64, interleaved=inter))
    base = dict(hidden_size=32, num_heads=4, num_kv_heads=2, head_dim=8)
    for more, error in ((dict(values="keys", value_dim=6), ValueError), (dict(values="keys", bias=True), ValueError),
                        (dict(sinks="two"), ValueError), (dict(values="q"), ValueError), (dict(gate=True, qk_norm="row"), NotImplementedError),
                        (dict(conv=3, sinks="one"), NotImplementedError), (dict(value_position=rope(4, 8)), ValueError),
                        (dict(value_position=rope(8, 8, True), position=rope(8, 8)), ValueError)):
        with pytest.raises(error):
            mixer_class("attention")(PartSpec("attention", dict(base, **more)), torch.float32)
    from xinfer_amd.parts import feed_forward_class
    moe = dict(hidden_size=32, intermediate_size=16, num_experts=3, top=4)
    with pytest.raises(ValueError):
        feed_forward_class("routed_experts")(PartSpec("routed_experts", moe), torch.float32)
    feed_forward_class("routed_experts")(PartSpec("routed_experts", dict(moe, identity=1)), torch.float32)
    with pytest.raises(ValueError):
        feed_forward_class("routed_experts")(PartSpec("routed_experts", dict(moe, top=1, correction=True)), torch.float32)


# ---- what fixes each rule of the plain implementation beside its text ------------------------------------------------
def test_norm_in_groups():
    x = torch.tensor([[3.0, 4.0, 30.0, 40.0]], dtype=torch.float64)
    w = torch.tensor([1.0, 2.0, 1.0, 10.0], dtype=torch.float64)
    r = math.sqrt(12.5)
    want = [3 / r, 2 * 4 / r, 3 / r, 10 * 4 / r]
    assert torch.allclose(plain.group_norm(x, 0.0, w, 2)[0], torch.tensor(want, dtype=torch.float64))
    assert torch.allclose(plain.group_norm(torch.zeros(1, 4) + 2.0, 5.0)[0], torch.full((4,), 2.0 / 3.0))


def test_the_convolution_sees_nothing_before_a_sequence():
    g = torch.Generator().manual_seed(2)
    h, w = torch.randn(6, 2, generator=g, dtype=torch.float64), torch.randn(2, 3, generator=g, dtype=torch.float64)
    out = plain.input_conv(h, w)
    assert torch.allclose(out[0], h[0] + w[:, 2] * h[0])
    assert torch.allclose(out[2], h[2] + w[:, 0] * h[0] + w[:, 1] * h[1] + w[:, 2] * h[2])


def test_what_a_query_sees():
    assert plain.window_seen(6, 2).sum(dim=1).tolist() == [1, 2, 2, 2, 2, 2] and bool(plain.window_seen(6, 2)[4, 3])
    assert not bool(plain.window_seen(6, 2)[4, 2]) and torch.equal(plain.window_seen(4, 1), torch.eye(4, dtype=torch.bool))
    assert [r.nonzero().flatten().tolist() for r in plain.chunk_seen(5, 3)] == [[0], [0, 1], [0, 1, 2], [3], [3, 4]]


def test_turning_and_sinks():
    x = torch.randn(5, 2, 12, dtype=torch.float64)
    a = plain.angles(100.0, 8, torch.arange(5))
    y = plain.turn_halves(x, a)
    assert torch.equal(y[0], x[0]) and torch.equal(y[..., 8:], x[..., 8:]) and torch.allclose(plain.turn_halves(y, -a), x)
    t = 3 * 100.0 ** (-2 / 8)                    # position 3, pair 1: dims 1 and 5
    assert torch.allclose(y[3, 0, 1], x[3, 0, 1] * math.cos(t) - x[3, 0, 5] * math.sin(t))
    assert torch.allclose(y[3, 0, 5], x[3, 0, 5] * math.cos(t) + x[3, 0, 1] * math.sin(t))
    q, k, v = torch.zeros(3, 1, 4), torch.zeros(3, 1, 4), torch.ones(3, 1, 2)      # every score is 0
    o = plain.softmax_heads(q, k, v, 1.0, plain.window_seen(3, 2), torch.zeros(1))
    assert torch.allclose(o[:, 0, 0], torch.tensor([1 / 2, 2 / 3, 2 / 3]))
    o = plain.softmax_heads(q, k, v, 1.0, plain.window_seen(3, 2), torch.tensor([math.log(6.0)]))
    assert torch.allclose(o[:, 0, 0], torch.tensor([1 / 7, 2 / 8, 2 / 8]))


def test_a_state_goes_on_where_a_portion_ended():
    g = torch.Generator().manual_seed(1)
    r = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
    x, B, C, d, a, D = r(9, 2, 5), r(9, 2, 3), r(9, 2, 3), torch.rand(9, 2, generator=g, dtype=torch.float64), r(2), r(2)
    y, S = plain.state_walk(x, B, C, d, a, D)
    y1, mid = plain.state_walk(x[:4], B[:4], C[:4], d[:4], a, D)
    y2, end = plain.state_walk(x[4:], B[4:], C[4:], d[4:], a, D, mid)
    assert torch.allclose(torch.cat([y1, y2]), y) and torch.allclose(end, S)
    assert torch.allclose(y[0, 1], d[0, 1] * (B[0, 1] @ C[0, 1]) * x[0, 1] + D[1] * x[0, 1])


def test_choice_by_corrected_scores_and_weights_without():
    z = torch.tensor([[2.0, 1.0, 0.0, -1.0]], dtype=torch.float64)
    s = torch.softmax(z, -1)[0]
    chosen, wt = plain.route(z, torch.eye(4, dtype=torch.float64), torch.tensor([-1.0, 0.0, 0.0, 0.5], dtype=torch.float64), 2)
    assert chosen.tolist() == [[3, 1]]
    assert torch.allclose(wt[0], torch.stack([s[3], s[1]]) / (s[3] + s[1]))
