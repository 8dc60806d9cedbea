"""Lopazen without a GPU: the plain equations against themselves (closed forms, cuts), configuration, tensors, registry."""
import numpy as np
import pytest

import lopazen_cases as lc
from flexllm_amd import hybrid, loader, lopazen, registry
from oracle import lopazen_ref as ref


def test_equations_do_not_depend_on_cuts():
    cfg = lc.mixed()
    w, toks = lc.weights(cfg, 1), lc.tokens(cfg, 60)
    whole = ref.Reference(cfg, w).run(toks)
    r = ref.Reference(cfg, w)
    parts = np.concatenate([r.run(toks[a:b]) for a, b in ((0, 1), (1, 3), (3, 40), (40, 60))])
    assert np.abs(whole - parts).max() < 1e-10


def test_temperature_steps():
    assert ref.temperature(0, 0.5, 4) == 1.0 and ref.temperature(2, 0.5, 4) == 1.0
    assert np.isclose(ref.temperature(3, 0.5, 4), 1.0 + 0.5 * np.log(2.0)) and ref.temperature(6, 0.5, 4) == ref.temperature(3, 0.5, 4)
    assert np.isclose(ref.temperature(7, 0.5, 4), 1.0 + 0.5 * np.log(3.0))


def test_sink_takes_part_in_the_sum():
    assert np.allclose(ref.sink_softmax(np.array([0.0])), 0.5)
    s = np.array([1.0, -2.0, 0.5])
    assert np.allclose(ref.sink_softmax(s), np.exp(s) / (1.0 + np.exp(s).sum()))
    assert np.allclose(ref.sink_softmax(np.array([-800.0, -900.0])), 0.0) and np.allclose(ref.sink_softmax(np.array([800.0, 800.0])), 0.5)


def test_values_are_keys_ahead_of_their_norm():
    cfg = lc.config([lc.layer(heads=1, kv_heads=1, dim=8, scale=0.5, coef=0.0)])
    w = lc.weights(cfg, 2)
    h = np.random.default_rng(3).standard_normal((1, 160))
    keys, values = ref.key_values(cfg["layers"][0]["mixer"], w, "l0.mix.", h, 1e-5)
    v = h @ w["l0.mix.k"].T + w["l0.mix.k.b"]
    assert np.allclose(values[0, 0], v) and np.allclose(keys[0, 0], v[0] / np.sqrt((v ** 2).mean() + 1e-5) * w["l0.mix.k.norm"])
    q = h @ w["l0.mix.q"].T + w["l0.mix.q.b"]
    s = (q[0] / np.sqrt((q ** 2).mean() + 1e-5) * w["l0.mix.q.norm"]) @ keys[0, 0] * 0.5
    out = ref.attention(cfg["layers"][0]["mixer"], w, "l0.mix.", h, 0, keys, values, 1e-5)
    assert np.allclose(out, (v / (1.0 + np.exp(-s))) @ w["l0.mix.o"].T)      # one key beside the sink


def test_order_of_runs():
    cfg = lc.config([lc.layer()] * 5, loop=(1, 3, 3))
    assert ref.layer_runs(cfg) == [(0, False), (1, False), (2, False), (1, True), (2, False), (1, True), (2, False), (3, False), (4, False)]
    assert ref.layer_runs(lc.config([lc.layer()] * 2)) == [(0, False), (1, False)]
    assert ref.layer_runs(lc.config([lc.layer()], loop=(0, 1, 2))) == [(0, False), (0, True)]


def test_loop_written_out():
    """Two passes over one layer: each with keys of its own, the embedding output added between them."""
    cfg = lc.config([lc.layer()], loop=(0, 1, 2))
    w, toks = lc.weights(cfg, 4), lc.tokens(cfg, 7)
    mx, eps = cfg["layers"][0]["mixer"], cfg["norm"]["eps"]
    first = w["embed"].astype(np.float64)[toks] * 3.0

    def once(x):
        h = ref.rms_norm(x, w["l0.norm1"], eps)
        return x + ref.attention(mx, w, "l0.mix.", h, 0, *ref.key_values(mx, w, "l0.mix.", h, eps), eps)
    x = once(once(first) + first)
    assert np.allclose(ref.Reference(cfg, w).run(toks), ref.rms_norm(x, w["final.norm"], eps) @ w["embed"].T)


def test_gelu():
    z = np.array([-30.0, -1.0, 0.0, 0.5, 30.0])
    assert np.allclose(ref.gelu(z), [0.0, -0.15880800939, 0.0, 0.345714, 30.0], atol=1e-6)


def test_descriptors():
    cfg = lc.mixed()
    d = [lopazen.layer_descriptor(i, ly) for i, ly in enumerate(cfg["layers"])]
    assert all(x["mixer"] == hybrid.MIX_SHARED_KV and x["sink"] == 1 for x in d)
    assert (d[0]["heads"], d[0]["kv_heads"], d[0]["dim"], d[0]["scale"], d[0]["temp_coef"], d[0]["temp_every"]) == (6, 2, 24, 0.2, 0.4, 16)
    assert d[0]["ff_kind"] == hybrid.FF_DENSE and d[0]["glu"] == hybrid.GLU_GELU and d[2]["ff_kind"] == hybrid.FF_NONE
    assert lopazen.loop_of(cfg) == (1, 3, 3) and lopazen.loop_of(dict(cfg, loop=None)) == (0, 0, 1)
    shapes = lopazen.tensor_shapes(cfg)
    assert shapes["l1.mix.k"] == (160, 160) and shapes["l2.mix.q.b"] == (80,) and "l2.norm2" not in shapes and "head" not in shapes
    bad = lc.layer()
    bad["mixer"]["vdim"] = 8
    for ly, text in ((dict(lc.layer(), type="other"), "unknown mixer"), (lc.layer(mlp=dict(kind="other")), "unknown feed-forward"), (bad, "vdim 8")):
        with pytest.raises(hybrid.ConfigError, match=text):
            lopazen.layer_descriptor(0, ly)
    for loop in ((0, 5, 2), (3, 2, 2), (-1, 2, 2), (0, 2, 0)):
        with pytest.raises(hybrid.ConfigError, match="cannot run"):
            lopazen.loop_of(lc.config([lc.layer()] * 4, loop=loop))


def test_every_field_and_every_tensor_has_its_place():
    from flexllm_amd._lib import HybridLayer, HybridLayerWeights
    cfg = lc.mixed()
    shapes = lopazen.tensor_shapes(cfg)
    fields, names = {n for n, _ in HybridLayer._fields_}, {n for n, _ in HybridLayerWeights._fields_}
    for i, ly in enumerate(cfg["layers"]):
        assert set(lopazen.layer_descriptor(i, ly)) <= fields
    grouped = hybrid.group_weights(cfg, lambda n: n, shapes)
    assert all(set(w) <= names for w in grouped["layers"])
    assert {n for w in grouped["layers"] for n in w.values()} | {"embed", "final.norm"} == set(shapes)
    assert grouped["head"] == grouped["embed"] == "embed"            # tied


def test_missing_and_misshapen_tensors():
    cfg = lc.config([lc.layer(mlp=lc.dense())])
    w = lc.weights(cfg, 1)
    with pytest.raises(loader.ParameterError, match="missing tensor l0.mix.k.b"):
        lopazen.Lopazen.from_tensors(cfg, {n: a for n, a in w.items() if n != "l0.mix.k.b"})
    for name in ("l0.mix.o", "l0.mix.q.norm", "l0.mlp.down"):
        with pytest.raises(loader.ParameterError, match=name + " has shape"):
            lopazen.Lopazen.from_tensors(cfg, dict(w, **{name: w[name][:-1]}))


def test_registry():
    assert "Lopazen" in registry.architectures() and registry.model_class("Lopazen") is lopazen.Lopazen
