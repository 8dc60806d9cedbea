"""Nifunex without a GPU: the plain equations against themselves (closed forms, cuts), configuration, tensors, files, slots."""
import json
import os

import numpy as np
import pytest

import nifunex_cases as nc
from flexllm_amd import loader, nifunex, registry
from flexllm_amd.slots import NoFreeSlot, SlotPool
from oracle import nifunex_ref as ref


def test_equations_do_not_depend_on_cuts():
    cfg = nc.mixed()
    w, toks = nc.weights(cfg, 1), nc.tokens(cfg, 60)
    whole = ref.Reference(cfg, w).run(toks)
    r = ref.Reference(cfg, w)
    parts = np.concatenate([r.run(toks[a:b]) for a, b in ((0, 1), (1, 3), (3, 40), (40, 60))])
    assert np.abs(whole - parts).max() < 1e-10


def test_recurrence_equals_the_sum_over_earlier_tokens():
    r = np.random.default_rng(2)
    q, k, v = r.standard_normal((9, 2, 5)), r.standard_normal((9, 2, 5)), r.standard_normal((9, 2, 4))
    la = -r.random((9, 2, 5))
    o = ref.gla_recurrence(q, k, v, la, np.zeros((2, 5, 4)))
    L = np.cumsum(la, 0)
    for t in range(9):
        for h in range(2):
            want = sum((q[t, h] * k[j, h] * np.exp(L[t, h] - L[j, h])).sum() * v[j, h] for j in range(t + 1))
            assert np.allclose(o[t, h], want)


def test_latent_scores_in_the_latent_space():
    """q . (W_uk c) = (W_uk^T q) . c: the form that attends over the cached rows."""
    r = np.random.default_rng(3)
    w_uk, c, q = r.standard_normal((6, 4)), r.standard_normal(4), r.standard_normal(6)
    assert np.isclose(q @ (w_uk @ c), (w_uk.T @ q) @ c)


def test_rotation_keeps_relative_places():
    rot = dict(base=100.0, dims=8, scaling=dict(factor=4.0, original=32, fast=4.0, slow=1.0))
    r = np.random.default_rng(4)
    a, b = r.standard_normal(8), r.standard_normal(8)
    s = [ref.rotate_pairs(a, p + 5, rot) @ ref.rotate_pairs(b, p, rot) for p in (0, 3, 40)]
    assert np.allclose(s, s[0])
    f, m = ref.yarn_frequencies(rot)
    plain, one = ref.yarn_frequencies(dict(base=100.0, dims=8))
    assert one == 1.0 and np.isclose(m, 0.1 * np.log(4.0) + 1.0)
    assert np.all(f <= plain + 1e-15) and np.all(f >= plain / 4.0 - 1e-15) and np.isclose(f[-1], plain[-1] / 4.0)


def test_window_edges():
    cfg = nc.config([nc.latent(window=4, heads=1)])
    w, toks = nc.weights(cfg, 5), nc.tokens(cfg, 12)
    base = ref.Reference(cfg, w).run(toks)[-1]
    for back, seen in ((3, True), (4, False)):
        t = list(toks)
        t[11 - back] = (t[11 - back] + 1) % cfg["vocab"]
        assert (np.abs(ref.Reference(cfg, w).run(t)[-1] - base).max() > 1e-6) == seen


def test_router():
    pick, wt = ref.route(np.array([0.0, 2.0, 2.0, -1.0]), 2)
    assert pick.tolist() == [1, 2] and np.allclose(wt, 0.5)
    g = ref.clamped_glu(np.array([5.0, -3.0]), np.array([-9.0, 9.0]), 2.0)
    assert np.allclose(g, [2.0 / (1 + np.exp(-3.404)) * -1.0, -3.0 / (1 + np.exp(5.106)) * 3.0])


def test_log_of_decay():
    cfg = nc.gla(heads=1, dim=4, vdim=3, tau=4.0)["mixer"]
    r = np.random.default_rng(6)
    w = {"a1": r.standard_normal((2, 6)), "a2": r.standard_normal((4, 2)), "a2.b": r.standard_normal(4)}
    h = r.standard_normal((3, 6))
    z = h @ w["a1"].T @ w["a2"].T + w["a2.b"]
    assert np.allclose(np.exp(ref.gla_decay_log(cfg, w, "", h))[:, 0], (1 / (1 + np.exp(-z))) ** 0.25)


def test_descriptors():
    cfg = nc.mixed()
    shapes = nifunex.tensor_shapes(cfg, 12)
    d = [nifunex.layer_descriptor(i, ly, shapes.__getitem__) for i, ly in enumerate(cfg["layers"])]
    assert d[0]["mixer"] == nifunex.MIX_GLA and d[0]["a_rank"] == 12 and d[0]["ff_kind"] == nifunex.FF_DENSE and d[0]["limit"] == 1.25
    assert d[1]["kv_from"] == -1 and d[1]["window"] == 33 and d[1]["yarn"] == 1 and d[1]["shared_ff"] == 56 and d[1]["shared_limit"] == 2.0
    assert d[2]["kv_from"] == 1 and d[2]["window"] == 9 and "shared_ff" not in d[2] and d[2]["top"] == 3
    assert d[3]["ff_kind"] == nifunex.FF_NONE and "yarn" not in d[4]
    assert "l2.mix.dkv" not in shapes and "l3.norm2" not in shapes and shapes["l1.mlp.shared.sg"] == (1, 160)
    bad = nc.config([dict(type="other", mixer=dict(heads=1, dim=1, vdim=1))])
    with pytest.raises(nifunex.ConfigError, match="unknown mixer"):
        nifunex.layer_descriptor(0, bad["layers"][0], shapes.__getitem__)
    with pytest.raises(nifunex.ConfigError, match="unknown feed-forward"):
        nifunex.layer_descriptor(0, nc.gla(mlp=dict(kind="other")), shapes.__getitem__)


def test_descriptor_fields_exist():
    from flexllm_amd._lib import HybridLayer, HybridLayerWeights
    cfg = nc.mixed()
    shapes = nifunex.tensor_shapes(cfg)
    fields = {n for n, _ in HybridLayer._fields_}
    for i, ly in enumerate(cfg["layers"]):
        assert set(nifunex.layer_descriptor(i, ly, shapes.__getitem__)) <= fields
    names = {n for n, _ in HybridLayerWeights._fields_}
    for w in nifunex.group_weights(cfg, lambda n: n, shapes)["layers"]:
        assert set(w) <= names
    used = {n for w in nifunex.group_weights(cfg, lambda n: n, shapes)["layers"] for v in w.values() for n in (v if isinstance(v, list) else [v])}
    assert used | {"embed", "head", "final.norm"} == set(shapes)      # every tensor has its place


def test_missing_and_misshapen_tensors():
    cfg = nc.config([nc.gla()])
    w = nc.weights(cfg, 1)
    with pytest.raises(loader.ParameterError, match="missing tensor l0.mix.a2.b"):
        nifunex.Nifunex.from_tensors(cfg, {n: a for n, a in w.items() if n != "l0.mix.a2.b"})
    with pytest.raises(loader.ParameterError, match="l0.mix.o has shape"):
        nifunex.Nifunex.from_tensors(cfg, dict(w, **{"l0.mix.o": w["l0.mix.o"][:-1]}))
    with pytest.raises(loader.ParameterError, match="rank"):
        nifunex.Nifunex.from_tensors(cfg, dict(w, **{"l0.mix.a1": w["l0.mix.a1"][:-1]}))


def test_safetensors_round_trip(tmp_path):
    r = np.random.default_rng(7)
    t = {"a": r.standard_normal((3, 5)).astype(np.float32), "b.c": r.integers(0, 65536, (4,), dtype=np.uint16), "i": np.arange(6, dtype=np.int32).reshape(2, 3)}
    path = str(tmp_path / "x.safetensors")
    loader.write_safetensors(path, t)
    back = loader.read_safetensors(path)
    assert set(back) == set(t) and all(np.array_equal(back[n], t[n]) and back[n].dtype == t[n].dtype for n in t)
    from safetensors import safe_open
    from safetensors.numpy import save_file
    with safe_open(path, framework="np") as f:
        assert set(f.keys()) == set(t) and np.array_equal(f.get_tensor("a"), t["a"])
    save_file({"a": t["a"], "i": t["i"]}, path)
    assert np.array_equal(loader.read_safetensors(path)["i"], t["i"])
    with open(path, "r+b") as f:
        f.truncate(os.path.getsize(path) - 1)
    with pytest.raises(loader.ParameterError):
        loader.read_safetensors(path)


def test_bf16_rounding():
    import torch
    a = np.concatenate([np.random.default_rng(8).standard_normal(1000).astype(np.float32), np.float32([0.0, -0.0, 1.0, 1.00390625, 3.3895e38])])
    want = torch.from_numpy(a).to(torch.bfloat16).to(torch.float32).numpy()
    assert np.array_equal(loader.from_bf16(loader.to_bf16(a)), want)


def test_registry(tmp_path):
    assert "Nifunex" in registry.architectures() and registry.model_class("Nifunex") is nifunex.Nifunex
    with pytest.raises(registry.UnknownModel, match="neither"):
        registry.load_model(str(tmp_path))
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Nothing"}))
    with pytest.raises(registry.UnknownModel, match="Nothing"):
        registry.load_model(str(tmp_path))


def test_slot_pool():
    started = []
    p = SlotPool(2, started.append)
    a, b = p.acquire("a"), p.slot("b")
    assert a != b and p.slot("a") == a and p.free == 0 and started == [a, b]
    with pytest.raises(NoFreeSlot):
        p.acquire("c")
    with pytest.raises(KeyError):
        p.acquire("a")
    p.release("a")
    assert "a" not in p and p.acquire("c") == a and started == [a, b, a]


def test_component_sources_exist():
    from flexllm_amd import build
    have = {os.path.basename(s)[:-4] for s in build.sources()}
    for srcs in build.COMPONENTS.values():
        assert set(srcs) <= have
