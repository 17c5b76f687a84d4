"""Fuvevik on the CPU: the configuration reader and its refusals, the model as data (which entry reads which cache), the
tensors a model asks for, and hand-worked cases of the plain implementation's pieces."""
import copy
import math

import numpy as np
import pytest

import fuvevik_configs as Z
import plain_fuvevik as P

import nanoinfer_amd  # noqa: F401
from nanoinfer_amd.config.fuvevik_config import FuvevikConfig
from nanoinfer_amd.config.model_config import ConfigError
from nanoinfer_amd.registry import architecture_of
from nanoinfer_amd.weights.loader import check_tensors, expected_tensors


def spec_of(cfg):
    arch = architecture_of(cfg)
    return arch.build_spec(arch.config_from_dict(cfg))


@pytest.mark.parametrize("name", sorted(Z.ALL))
def test_configuration_round_trip_and_spec(name):
    cfg = Z.ALL[name]
    typed = FuvevikConfig.from_dict(cfg)
    assert FuvevikConfig.from_dict(typed.to_dict()) == typed
    spec = spec_of(cfg)
    assert len(spec.blocks) == len(spec.order) == len(cfg["layers"])
    for i, (layer, run, block) in enumerate(zip(cfg["layers"], spec.order, spec.blocks)):
        src = layer["mixer"].get("kv_from")
        assert run.block == i and run.cache == (i if src is None else src) and run.writes_cache == (src is None)
        assert ("ffn" in block.parts) == (layer["mlp"] is not None) == ("ffn_norm" in block.parts) == ("ffn_link" in block.parts)
        assert block.kind == "linked_streams" and block.params["streams"] == cfg["streams"]
        temp = layer["mixer"].get("q_temp") or {"coef": None, "every": None}
        assert block.mixer.params["temp_coef"] == temp["coef"] and block.mixer.params["temp_every"] == temp["every"]


def test_tensors_of_a_model():
    names = expected_tensors(spec_of(Z.SHARED_KV))
    assert names["embed"] == (97, 64) and names["final.norm"] == (64,) and "head" not in names and "embed.norm" not in names
    assert names["l0.mix.q"] == (64, 64) and names["l0.mix.k"] == (32, 64) and names["l0.mix.v"] == (16, 64)
    assert names["l0.mix.q.norm"] == (16,) and names["l0.mix.k.norm"] == (16,) and names["l0.mix.sink"] == (4,)
    assert names["l0.mix.g"] == (32, 64) and names["l0.mix.o"] == (64, 32)
    for gone in ("l2.mix.k", "l2.mix.v", "l2.mix.k.norm", "l3.mix.k", "l1.norm2", "l1.hc2.in", "l0.mlp.router", "l0.mlp.gate"):
        assert gone not in names
    assert names["l2.mix.q"] == (32, 64) and names["l3.mix.g"] == (48, 64) and names["l0.mlp.up"] == (96, 64) and names["l4.mlp.down"] == (64, 33)
    for hc in ("l0.hc1", "l0.hc2", "l1.hc1"):
        assert names[hc + ".in"] == (4,) and names[hc + ".out"] == (4,) and names[hc + ".mix"] == (4, 4)
    assert names["l2.mlp.router"] == (5, 64) and names["l2.mlp.correction"] == (5,) and names["l2.mlp.e3.down"] == (64, 16)
    assert "l2.mlp.e4.down" not in names and "l2.mlp.shared.gate" not in names
    moe = expected_tensors(spec_of(Z.MOE_ONLY))
    assert moe["l0.mlp.shared.gate"] == (40, 56) and moe["l0.mlp.router"] == (15, 56) and moe["l0.mlp.e11.up"] == (24, 56)
    # the tensors of a sublayer that a layer does not have may be there all the same
    import torch
    spec = spec_of(Z.ATTN_ONLY)
    held = {n: torch.zeros(s) for n, s in expected_tensors(spec).items()}
    held.update({"l0.norm2": torch.zeros(64), "l0.hc2.in": torch.zeros(2), "l0.hc2.out": torch.zeros(2), "l0.hc2.mix": torch.zeros(2, 2)})
    assert set(check_tensors(spec, held)) == set(expected_tensors(spec))


def test_refusals():
    def broken(edit, base=Z.MIXED):
        cfg = copy.deepcopy(base)
        edit(cfg)
        with pytest.raises(ConfigError):
            FuvevikConfig.from_dict(cfg)

    broken(lambda c: c["layers"][0].update(type="conv"))
    broken(lambda c: c["layers"][1]["mixer"].update(kv_heads=4))             # 6 heads on 4
    broken(lambda c: c["layers"][1]["mixer"]["q_temp"].update(every=0))
    broken(lambda c: c["layers"][1]["mixer"]["q_temp"].pop("coef"))
    broken(lambda c: c["layers"][3]["mixer"].update(kv_from=3))              # not an earlier layer
    broken(lambda c: c["layers"][3]["mixer"].update(kv_from=0))              # other sizes than the layer it reads
    broken(lambda c: c["layers"][4]["mixer"].update(kv_from=3))              # a layer that makes no keys
    broken(lambda c: c["layers"][1]["mlp"]["router"].update(top=11))         # 11 of 8 + 2
    broken(lambda c: c["layers"][1]["mlp"]["router"].update(identity=-1))
    broken(lambda c: c["layers"][1]["mlp"].update(kind="gated"))
    broken(lambda c: c["layers"][1]["mlp"]["expert"].pop("limit"))
    broken(lambda c: c["layers"][1]["mlp"]["shared"].pop("limit"))
    broken(lambda c: c["layers"][0]["mlp"].pop("ff"))
    broken(lambda c: c.pop("streams"))
    broken(lambda c: c.update(streams=0))
    broken(lambda c: c.pop("norm"))
    broken(lambda c: c.update(layers=[]))


def test_a_model_has_one_number_of_streams():
    """Blocks hand the streams on among themselves: one of another number, or a block over one stream beside them, is an
    error when the model is put together, not at its first step."""
    from nanoinfer_amd.engine.model import Model

    class FakeBlock:
        def __init__(self, streams):
            if streams is not None:
                self.streams = streams

        def cache_need(self):
            return None

    class FakeRuntime:
        dtype = None

    import nanoinfer_amd.engine.model as M
    real_part, real_get = M.build_part, M.get_part
    M.build_part = lambda *a: object()
    try:
        for blocks, ok in (((2, 2), True), ((2, 3), False), ((None, None), True), ((2, None), False)):
            made = iter(blocks)
            M.get_part = lambda family, kind: (lambda spec, tensors, rt: FakeBlock(next(made)))
            spec = spec_of(Z.MANY_STREAMS)
            if ok:
                Model(spec, {}, FakeRuntime())
            else:
                with pytest.raises(ValueError, match="streams"):
                    Model(spec, {}, FakeRuntime())
    finally:
        M.build_part, M.get_part = real_part, real_get


def test_the_sinusoid_by_hand():
    s = P.sinusoid(np.array([0, 3]), 6)
    assert np.allclose(s[0], [0, 1, 0, 1, 0, 1])
    for i in range(3):
        a = 3 * 10000.0 ** (-2 * i / 6)
        assert math.isclose(s[1, 2 * i], math.sin(a)) and math.isclose(s[1, 2 * i + 1], math.cos(a))
    assert np.allclose(P.sinusoid(np.array([5]), 5), P.sinusoid(np.array([5]), 10)[:, :5] * 0 + [
        [math.sin(5), math.cos(5), math.sin(5 * 10000 ** -.4), math.cos(5 * 10000 ** -.4), math.sin(5 * 10000 ** -.8)]])


def test_the_streams_by_hand():
    x = np.array([[[1.0, 2.0]], [[10.0, 20.0]]])                       # two streams, one token, width two
    w = {"h.in": np.array([0.5, 2.0]), "h.out": np.array([3.0, -1.0]), "h.mix": np.array([[1.0, 0.1], [0.0, 2.0]])}
    assert np.allclose(P.sublayer_input(x, w, "h."), [[20.5, 41.0]])
    y = np.array([[100.0, 0.0]])
    # mix is indexed [from, to]: the first new stream is the first old one, the second a tenth of it plus twice the second
    assert np.allclose(P.sublayer_output(x, y, w, "h."), [[[301.0, 2.0]], [[0.1 + 20.0 - 100.0, 0.2 + 40.0]]])


def test_the_norm_stored_around_zero_by_hand():
    got = P.norm(np.array([[3.0, 4.0]]), np.array([0.0, 1.0]), 0.5)
    r = math.sqrt(12.5 + 0.5)
    assert np.allclose(got, [[3.0 / r, 8.0 / r]])


def test_the_query_factor_by_hand():
    t = P.temperature(np.array([0, 8, 9, 10, 18, 19, 99]), {"coef": 0.5, "every": 10})
    steps = [0, 0, 1, 1, 1, 2, 10]
    assert np.allclose(t, [1 + 0.5 * math.log(s + 1) for s in steps])
    assert np.allclose(P.temperature(np.array([0, 7]), None), 1.0)
    assert np.allclose(P.temperature(np.array([0, 1]), {"coef": 1.0, "every": 1}), [1 + math.log(2), 1 + math.log(3)])


def test_softmax_with_a_sink_by_hand():
    p = P.sink_softmax(np.zeros((3, 3)), 0.0)                         # the sink weighs like a key
    assert np.allclose(p, [[1 / 2, 0, 0], [1 / 3, 1 / 3, 0], [1 / 4, 1 / 4, 1 / 4]])
    assert np.allclose(P.sink_softmax(np.zeros((3, 3)), math.log(2.0))[2], [1 / 5] * 3)
    assert np.allclose(P.sink_softmax(np.zeros((2, 2)), -1e9)[1], [.5, .5])
    assert np.allclose(P.sink_softmax(np.full((2, 2), -800.0), 700.0), 0.0)


def test_the_router_by_hand():
    # four experts and two that give their input back; shares of the softmax (as logits below) plus correction
    s = np.array([0.4, 0.1, 0.05, 0.2, 0.15, 0.1])
    w = {"l0.mlp.router": np.diag(np.log(s) + 3.0) @ np.ones((6, 6)) / 6.0, "l0.mlp.correction": np.array([-0.35, 0.0, 0.3, 0.0, 0.0, 0.0])}
    mlp = {"router": {"experts": 4, "identity": 2, "top": 3}}
    h = np.ones((1, 6))
    margins = np.full(1, np.inf)
    chosen, weights = P.route(h, mlp, w, "l0.", margins)
    assert chosen.tolist() == [[2, 3, 4]]                              # .35 .2 .15; the largest share, at .05 now, is left out
    assert np.allclose(weights, [np.array([0.05, 0.2, 0.15]) / 0.4])    # the weights never see the correction
    assert math.isclose(margins[0], (0.15 - 0.1) / 0.15)


def test_identity_experts_and_the_shared_expert_by_hand():
    d = 2
    w = {"l0.mlp.router": np.zeros((3, d)), "l0.mlp.correction": np.array([0.0, 1.0, 0.5])}
    for e in ("e0", "shared"):
        w.update({f"l0.mlp.{e}.gate": np.eye(d), f"l0.mlp.{e}.up": np.zeros((d, d)), f"l0.mlp.{e}.down": np.eye(d)})
    mlp = {"router": {"experts": 1, "identity": 2, "top": 2}, "expert": {"limit": 9.0}}
    h = np.array([[3.0, -1.0]])
    assert np.allclose(P.routed(h, mlp, w, "l0."), h)                  # both chosen outputs give the input back
    mlp["router"]["top"] = 3
    g = h / (1 + np.exp(-1.702 * h))                                   # an expert with identity matrices and no up values
    assert np.allclose(P.routed(h, mlp, w, "l0."), 2 * h / 3 + g / 3)
    mlp["shared"] = {"limit": 2.0}
    capped = np.minimum(h, 2.0)
    assert np.allclose(P.routed(h, mlp, w, "l0."), 2 * h / 3 + g / 3 + capped / (1 + np.exp(-1.702 * capped)))


def test_an_expert_and_the_dense_feed_forward_by_hand():
    w = {"e.gate": np.array([[1.0, 0.0], [0.0, 1.0]]), "e.up": np.array([[0.0, 1.0], [1.0, 0.0]]), "e.down": np.array([[1.0, 1.0]])}
    h = np.array([[3.0, -0.5]])                                   # gates 3 -> 2 (capped), -0.5; ups -0.5, 3 -> 2 (capped)
    g0, g1 = 2.0, -0.5
    want = g0 / (1 + math.exp(-1.702 * g0)) * (-0.5 + 1) + g1 / (1 + math.exp(-1.702 * g1)) * (2.0 + 1)
    assert np.allclose(P.expert(h, w, "e.", 2.0), [[want]])
    w = {"mlp.up": np.array([[1.0, 1.0], [1.0, -1.0]]), "mlp.down": np.array([[1.0, 10.0]])}
    assert np.allclose(P.dense(np.array([[1.0, 3.0]]), w, ""), [[16.0]])


def random_weights(cfg, rng):
    w = {}
    for name, shape in expected_tensors(spec_of(cfg)).items():
        std = 0.12 if len(shape) > 1 else 0.1
        centre = 1.0 if name.endswith((".q.norm", ".k.norm", ".out")) else 0.4 if name.endswith((".in", "hc1.mix", "hc2.mix")) else 0.0
        w[name] = rng.normal(size=shape) * std + centre
    return w


def test_every_mechanism_weighs_in_the_plain_model():
    """With a tensor of each mechanism moved (or a switch turned) the plain logits move by far more than any tolerance."""
    rng = np.random.default_rng(0)
    cfg0 = Z.MIXED
    w = random_weights(cfg0, rng)
    toks = [int(t) for t in rng.integers(0, 131, size=90)]
    want = P.forward(cfg0, w, toks)

    def moved(weights=None, cfg=None):
        got = P.forward(cfg or cfg0, weights or w, toks)
        return float(np.abs(got - want).max() / np.abs(want).max())

    for key in ("l0.mix.o", "l1.mix.o", "l3.mix.o", "l2.mix.v", "l1.mlp.shared.down", "l2.mlp.router", "l3.mix.q", "l1.mix.v", "l0.mlp.down",
                "l0.hc1.in", "l4.hc2.out", "l2.hc1.mix"):
        dead = dict(w)
        dead[key] = np.zeros_like(w[key])
        assert moved(dead) > 3e-3, key
    for key, value in (("l1.mix.sink", 3.0), ("l4.mix.sink", 3.0), ("l1.mix.g", 2.0), ("l4.mix.g", 2.0), ("l1.mix.q.norm", 2.0),
                       ("l1.mix.k.norm", 2.0), ("l0.norm1", 2.0), ("l2.norm2", 2.0), ("final.norm", 2.0)):
        other = dict(w)
        other[key] = w[key] + value * (np.arange(w[key].size).reshape(w[key].shape) % 2)
        assert moved(other) > 1e-3, key
    turned = dict(w)
    turned["l1.hc2.mix"] = w["l1.hc2.mix"].T                           # [to, from] instead of [from, to]
    assert moved(turned) > 1e-3
    other = dict(w)
    other["l1.mlp.correction"] = w["l1.mlp.correction"] + np.array([2.0, 0, 0, 0, 0, 0, -2.0, 0, 0, 1.0])
    assert moved(other) > 1e-3
    for edit in (lambda c: c["layers"][1]["mixer"]["q_temp"].update(every=17), lambda c: c["layers"][0]["mixer"]["q_temp"].update(coef=0.8),
                 lambda c: c["layers"][3]["mixer"].pop("q_temp"), lambda c: c["layers"][2]["mixer"].update(scale=0.1),
                 lambda c: c["layers"][1]["mlp"]["expert"].update(limit=0.1), lambda c: c["layers"][2]["mlp"]["shared"].update(limit=0.05),
                 lambda c: c["layers"][4]["mlp"]["router"].update(top=3), lambda c: c["norm"].update(eps=0.1)):
        cfg = copy.deepcopy(cfg0)
        edit(cfg)
        assert moved(cfg=cfg) > 1e-4
