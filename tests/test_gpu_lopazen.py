"""Lopazen on the GPU against the plain statement of its equations (oracle/lopazen_ref.py): each mechanism alone, sizes of
many kinds, prompts against decoding and portions, slots used again, far keys, the sink, loops, long decoding, generation."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import lopazen_cases as lc
import nifunex_cases as nc
from oracle import lopazen_ref, nifunex_ref

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
BOTH = pytest.mark.parametrize("dtype", ["float32", "bfloat16"])


def model(cfg, w, dtype, max_pos=512, slots=1):
    from flexllm_amd.lopazen import Lopazen
    return Lopazen.from_tensors(cfg, w, dtype=dtype, max_pos=max_pos, slots=slots)


def run(m, toks, cuts):
    """Logits of every token, fed in portions of the given sizes (the last one repeats)."""
    key = object()
    s = m.pool.acquire(key)
    out, p, i = [], 0, 0
    while p < len(toks):
        c = min(cuts[min(i, len(cuts) - 1)], len(toks) - p)
        out.append(m.step(s, toks[p:p + c], range(c)))
        p += c
        i += 1
    m.check()
    m.pool.release(key)
    return np.concatenate(out)


def expect(cfg, w, toks):
    return lopazen_ref.Reference(cfg, w).run(toks)


def close(got, want, dtype, what=""):
    assert np.isfinite(got).all(), what
    e = lc.rel_err(got, want)
    assert e.max() < lc.LIMIT[dtype], "%s: error %.3g at place %d (mean %.3g)" % (what, e.max(), e.argmax(), e.mean())


ALONE = {
    "one layer": lc.config([lc.layer()]),
    "one head": lc.config([lc.layer(heads=1, kv_heads=1)]),
    "a key head per query head": lc.config([lc.layer(heads=4, kv_heads=4, dim=32)]),
    "one key head": lc.config([lc.layer(heads=6, kv_heads=1, dim=64)]),
    "two heads per key head": lc.config([lc.layer(heads=6, kv_heads=3, dim=48)]),
    "eight heads per key head": lc.config([lc.layer(heads=16, kv_heads=2, dim=16)]),
    "seven heads per key head": lc.config([lc.layer(heads=7, kv_heads=1, dim=40)]),
    "heads of 8": lc.config([lc.layer(dim=8, scale=0.4)]),
    "heads of 20": lc.config([lc.layer(heads=4, dim=20)]),
    "heads of 7": lc.config([lc.layer(heads=3, kv_heads=3, dim=7, scale=0.5)]),
    "heads of 72": lc.config([lc.layer(heads=2, kv_heads=1, dim=72, scale=0.12)]),
    "heads of 128": lc.config([lc.layer(heads=4, kv_heads=2, dim=128, scale=0.09)]),
    "heads of 160": lc.config([lc.layer(heads=2, kv_heads=2, dim=160, scale=0.08)]),
    "heads of 256": lc.config([lc.layer(heads=4, kv_heads=1, dim=256, scale=0.06)]),
    "heads beyond the matrix kernel": lc.config([lc.layer(heads=4, kv_heads=1, dim=264, scale=0.06)]),
    "heads of 500": lc.config([lc.layer(heads=2, kv_heads=1, dim=500, scale=0.045)]),
    "a temperature period of one": lc.config([lc.layer(coef=0.3, every=1)]),
    "no temperature": lc.config([lc.layer(coef=0.0)]),
    "a strong temperature": lc.config([lc.layer(coef=3.0, every=10, scale=0.05)]),
    "a negative scale": lc.config([lc.layer(scale=-0.3)]),
    "plain embedding": lc.config([lc.layer()], embed_scale=1.0),
    "feed-forward": lc.config([lc.layer(mlp=lc.dense(100))]),
    "feed-forward of odd size": lc.config([lc.layer(mlp=lc.dense(33))], width=64),
    "vectors of some length": lc.config([lc.layer(mlp=lc.dense(3000))], width=64),
    "long vectors": lc.config([lc.layer(mlp=lc.dense(8300))], width=64),
    "vectors of the greatest length": lc.config([lc.layer(mlp=lc.dense(15360))], width=64),
    "a large epsilon": lc.config([lc.layer(mlp=lc.dense())], eps=0.5),
    "one layer twice": lc.config([lc.layer(mlp=lc.dense())], loop=(0, 1, 2)),
    "all layers, four times": lc.config([lc.layer(mlp=lc.dense()), lc.layer(heads=2, dim=16)], loop=(0, 2, 4)),
    "the first layer again": lc.config([lc.layer(), lc.layer(heads=2, dim=16)], loop=(0, 1, 3)),
    "the last layer again": lc.config([lc.layer(), lc.layer(heads=2, dim=16)], loop=(1, 2, 3)),
    "a loop of no layers": lc.config([lc.layer(), lc.layer(heads=2, dim=16)], loop=(1, 1, 3)),
    "odd width and vocabulary": lc.config([lc.layer(mlp=lc.dense(33)), lc.layer(heads=2, dim=12)], width=90, vocab=131, loop=(0, 2, 2)),
    "no loop at all": dict(lc.config([lc.layer(), lc.layer()]), loop=None),
    "everything": lc.mixed(),
}


@BOTH
@pytest.mark.parametrize("name", list(ALONE))
def test_mechanism(name, dtype):
    cfg = ALONE[name]
    ref_cfg = dict(cfg, loop=cfg["loop"] or dict(start=0, stop=0, times=1))
    w = lc.weights(cfg, 3)
    toks = lc.tokens(cfg, 90)
    want = expect(ref_cfg, w, toks)
    m = model(cfg, w, dtype)
    close(run(m, toks, [90]), want, dtype, "whole prompt")
    close(run(m, toks, [70, 1]), want, dtype, "decoded")
    m.close()


@BOTH
def test_residual_after_every_layer_run(dtype):
    cfg = lc.mixed()
    w, toks = lc.weights(cfg, 4), lc.tokens(cfg, 40)
    trace = []
    lopazen_ref.Reference(cfg, w).run(toks, trace)
    m = model(cfg, w, dtype)
    assert m.layer_runs == len(trace) == 8
    for n in (40, 5):                                      # both schedules
        slot = m.pool.acquire(n)
        _, got = m.step(slot, toks[:n], [n - 1], layers=True)
        m.pool.release(n)
        for i, ref in enumerate(trace):
            err = np.abs(got[i] - ref[:n]).max() / np.sqrt((ref ** 2).mean())
            assert err < (2e-5 if dtype == "float32" else 8e-2), "run %d, %d tokens: %.3g" % (i, n, err)
    m.close()


@BOTH
@pytest.mark.parametrize("cuts", [[1], [2], [3, 2], [7, 9, 8], [16], [17, 1, 64], [63, 65, 2], [64], [129, 2]])
def test_portions(cuts, dtype):
    cfg = lc.mixed()
    w, toks = lc.weights(cfg, 5), lc.tokens(cfg, 200)
    m = model(cfg, w, dtype)
    close(run(m, toks, cuts), expect(cfg, w, toks), dtype, str(cuts))
    m.close()


def test_prompt_equals_decoding():
    cfg = lc.mixed()
    w, toks = lc.weights(cfg, 6), lc.tokens(cfg, 150)
    m = model(cfg, w, "float32")
    close(run(m, toks, [150]), run(m, toks, [1]), "float32")
    m.close()


@BOTH
def test_long_prompt_and_long_decoding(dtype):
    cfg = lc.config([lc.layer(heads=4, kv_heads=2, dim=64, scale=0.12, every=100, mlp=lc.dense()), lc.layer(heads=4, kv_heads=1, dim=32)], loop=(0, 1, 2))
    w, toks = lc.weights(cfg, 7), lc.tokens(cfg, 2300)
    want = expect(cfg, w, toks[:900])
    m = model(cfg, w, dtype, max_pos=2300)
    close(run(m, toks[:900], [900]), want, dtype, "prompt of 900")
    close(run(m, toks[:900], [500, 1]), want, dtype, "400 decoded tokens")
    slot = m.pool.acquire(0)                               # many rows per split
    m.step(slot, toks[:2290])
    got = np.concatenate([m.step(slot, toks[2290 + i:2291 + i], [0]) for i in range(10)])
    close(got, expect(cfg, w, toks)[2290:], dtype, "behind a prompt of 2290")
    m.close()


def outstanding(cfg, w, asks=7, key=11):
    """Makes every head of a one-layer model's query of token `asks` point at the key of token `key`; returns both and tokens
    whose keys that query hardly sees."""
    mx = cfg["layers"][0]["mixer"]
    r = np.random.default_rng(3)
    w["l0.mix.q.b"][:], w["l0.mix.q.norm"][:], w["l0.mix.k.norm"][:] = 0.0, 1.0, 1.0
    h = lopazen_ref.rms_norm(w["embed"] * cfg["embedding"]["scale"], w["l0.norm1"], cfg["norm"]["eps"])
    _, k, _ = lc.split_qk(cfg, w)
    want = r.standard_normal((cfg["vocab"], mx["heads"], mx["dim"]))
    for n in range(mx["heads"]):
        want[asks, n] = k[key, n // (mx["heads"] // mx["kv_heads"])]
    w["l0.mix.q"] = lc.round_bf16((np.linalg.pinv(h) @ want.reshape(cfg["vocab"], -1)).T)
    q, k, _ = lc.split_qk(cfg, w)
    s = q[asks, 0] @ k[:, 0].T * mx["scale"]
    assert s.argmax() == key
    return asks, key, [int(t) for t in np.argsort(s)[:20] if t not in (asks, key)]


@BOTH
@pytest.mark.parametrize("heads,kv_heads,dim", [(1, 1, 32), (4, 1, 64), (3, 1, 128)])
def test_far_keys(heads, kv_heads, dim, dtype):
    """One key whose score stands out, at the borders of tiles and splits, read by a prompt's last token, by a decoded one
    and by one in a short portion; also as the newest row, and in the step that stores it."""
    cfg = lc.config([lc.layer(heads=heads, kv_heads=kv_heads, dim=dim, scale=12.0 / dim, coef=0.0)], vocab=120)
    w = lc.weights(cfg, 10)
    asks, key, fill = outstanding(cfg, w)
    m = model(cfg, w, dtype, max_pos=1200)
    rng = np.random.default_rng(0)
    for n, places in ((200, (0, 1, 31, 32, 63, 64, 65, 127, 128, 197, 198, 199)), (1100, (0, 511, 512, 1023, 1024, 1098))):
        base = rng.choice(fill, n + 1).tolist()
        base[n] = asks
        without = expect(cfg, w, base)[-1:]
        for p in places:
            toks = list(base)
            toks[p] = key
            want = expect(cfg, w, toks)[-1:]
            assert nc.rel_err(want, without)[0] > 0.2      # the case is sharp
            for cuts in ([n + 1], [n, 1], [n - 1, 2], [n - 20, 21]):
                close(run(m, toks, cuts)[-1:], want, dtype, "n=%d place %d cuts %s" % (n, p, cuts))
    m.close()


@BOTH
def test_future_keys_are_not_seen(dtype):
    """A key that stands out right behind a query changes nothing for it, in a prompt and in a step of few tokens."""
    cfg = lc.config([lc.layer(heads=2, kv_heads=1, dim=32, scale=0.4, coef=0.0)], vocab=120)
    w = lc.weights(cfg, 11)
    asks, key, fill = outstanding(cfg, w)
    m = model(cfg, w, dtype)
    for n in (5, 62, 63, 64, 100):
        toks = (fill * 10)[:n] + [asks, key, asks]
        want = expect(cfg, w, toks)
        assert nc.rel_err(want[n:n + 1], want[n + 2:n + 3])[0] > 0.2
        for cuts in ([n + 3], [n, 3], [n, 1], [n, 2]):
            close(run(m, toks, cuts), want, dtype, "n=%d cuts %s" % (n, cuts))
    m.close()


@BOTH
@pytest.mark.parametrize("sign", [-1.0, 1.0])
def test_sink(sign, dtype):
    """Scores that are all far below (above) the sink's, so that hardly anything (nearly everything) comes through."""
    cfg = lc.config([lc.layer(heads=2, kv_heads=2, dim=32, scale=0.2, coef=0.0)], vocab=90)
    w = lc.weights(cfg, 12)
    r = np.random.default_rng(1)
    w["embed"] = lc.round_bf16(0.3 * (np.ones((1, 160)) + 0.3 * r.standard_normal((90, 160))))      # tokens that resemble each other
    w["l0.mix.q"], w["l0.mix.q.b"] = lc.round_bf16(sign * w["l0.mix.k"]), lc.round_bf16(sign * w["l0.mix.k.b"])
    w["l0.mix.q.norm"][:], w["l0.mix.k.norm"][:] = 1.0, 1.0
    w["l0.norm1"][:] = 1.0
    toks = lc.tokens(cfg, 150)
    trace = []
    lopazen_ref.Reference(cfg, w).run(toks, trace)
    x0 = w["embed"][toks] * 3.0
    share = np.sqrt(((trace[0] - x0) ** 2).mean())          # what attention adds
    m = model(cfg, w, dtype)
    for n in (150, 1, 6):
        slot = m.pool.acquire(n)
        _, got = m.step(slot, toks[:n], [n - 1], layers=True)
        m.pool.release(n)
        added, want = got[0] - x0[:n], trace[0][:n] - x0[:n]
        tol = 1e-3 if dtype == "float32" else 3e-2
        assert np.abs(added - want).max() <= tol * np.abs(want).max() + 1e-6, "%d tokens" % n
    # without the sink the outputs would be of the values' size whatever the scores are
    values = np.sqrt(((lc.split_qk(cfg, w)[2][toks].reshape(150, -1) @ w["l0.mix.o"].T) ** 2).mean())
    assert share < 0.5 * values if sign < 0 else share > 0.8 * values
    close(run(m, toks, [100, 1]), expect(cfg, w, toks), dtype, "decoded")
    m.close()


@BOTH
def test_temperature_steps(dtype):
    """Places around the steps of the temperature, which change the outputs visibly."""
    cfg = lc.config([lc.layer(heads=2, kv_heads=1, dim=32, scale=0.15, coef=1.5, every=13)], vocab=90)
    w, toks = lc.weights(cfg, 13), lc.tokens(cfg, 70)
    want = expect(cfg, w, toks)
    late = dict(cfg, layers=[lc.layer(heads=2, kv_heads=1, dim=32, scale=0.15, coef=1.5, every=14)])
    off = nc.rel_err(expect(late, w, toks), want)
    assert off[12] > 0.1 and off[:12].max() < 1e-9          # position 12 is the first that has passed a period
    m = model(cfg, w, dtype)
    for cuts in ([70], [1], [12, 1], [13, 2]):
        close(run(m, toks, cuts), want, dtype, str(cuts))
    m.close()


@BOTH
def test_biases_that_cancel_the_projection(dtype):
    """Biases as large as what they are added to: they have to be in before anything is rounded."""
    cfg = lc.config([lc.layer(heads=4, kv_heads=2, dim=32)], vocab=90)
    w = lc.weights(cfg, 14)
    r = np.random.default_rng(2)
    w["embed"] = lc.round_bf16(0.3 * (np.ones((1, 160)) + 0.2 * r.standard_normal((90, 160))))
    h = lopazen_ref.rms_norm(w["embed"] * 3.0, w["l0.norm1"], 1e-5).mean(0)
    for n in ("q", "k"):
        w["l0.mix.%s.b" % n] = lc.round_bf16(-(w["l0.mix.%s" % n] @ h))
    toks = lc.tokens(cfg, 80)
    m = model(cfg, w, dtype)
    want = expect(cfg, w, toks)
    close(run(m, toks, [80]), want, dtype)
    close(run(m, toks, [60, 1]), want, dtype)
    m.close()


@BOTH
def test_slots(dtype):
    """Sequences in several slots, interleaved, and a slot that is used again, equal a sequence alone."""
    cfg = lc.mixed()
    w = lc.weights(cfg, 15)
    m = model(cfg, w, dtype, slots=2)
    a, b, c = lc.tokens(cfg, 120, 1), lc.tokens(cfg, 61, 2), lc.tokens(cfg, 40, 3)
    want = {n: expect(cfg, w, t) for n, t in (("a", a), ("b", b), ("c", c))}
    sa, sb = m.pool.acquire("a"), m.pool.acquire("b")
    got_a, got_b = [m.step(sa, a[:50], range(50))], [m.step(sb, b[:3], range(3))]
    got_a.append(m.step(sa, a[50:52], range(2)))
    got_b.append(m.step(sb, b[3:], range(58)))
    m.pool.release("b")
    sc = m.pool.acquire("c")
    assert sc == sb and m.length(sc) == 0
    got_c = [m.step(sc, c[:1], [0]), m.step(sc, c[1:], range(39))]
    got_a += [m.step(sa, a[52 + i:53 + i], [0]) for i in range(68)]
    for n, g in (("a", got_a), ("b", got_b), ("c", got_c)):
        close(np.concatenate(g), want[n], dtype, n)
    m.close()


def test_first_tokens():
    cfg = lc.mixed()
    w = lc.weights(cfg, 16)
    m = model(cfg, w, "float32")
    for n in (1, 2, 3, 8, 9):
        toks = lc.tokens(cfg, n, n)
        close(run(m, toks, [n]), expect(cfg, w, toks), "float32", "%d tokens" % n)
    m.close()


def test_many_pieces():
    """More tokens in one call than the library takes at a time."""
    cfg = lc.config([lc.layer(heads=2, kv_heads=1, dim=16)], width=64, vocab=80, loop=(0, 1, 2))
    w, toks = lc.weights(cfg, 17), lc.tokens(cfg, 4200)
    want = expect(cfg, w, toks)
    m = model(cfg, w, "bfloat16", max_pos=4200)
    slot = m.pool.acquire(0)
    places = [0, 4094, 4095, 4096, 4097, 4199]
    close(m.step(slot, toks, places), want[places], "bfloat16")
    m.close()


class LoopedNifunex(nifunex_ref.Reference):
    """Nifunex layers in the loop of the layer decoder."""

    def __init__(self, cfg, weights, loop):
        self.again = []
        order, cfg = lopazen_ref.layer_runs(dict(cfg, loop=dict(zip(("start", "stop", "times"), loop)))), dict(cfg)
        layers, w, latest = [], {n: a for n, a in weights.items() if not n.startswith("l")}, {}
        for r, (i, again) in enumerate(order):
            ly = dict(cfg["layers"][i], mixer=dict(cfg["layers"][i]["mixer"]))
            if ly["mixer"].get("kv_from") is not None:
                ly["mixer"]["kv_from"] = latest[ly["mixer"]["kv_from"]]
            latest[i] = r
            layers.append(ly)
            w.update({"l%d.%s" % (r, n.split(".", 1)[1]): a for n, a in weights.items() if n.startswith("l%d." % i)})
            self.again.append(again)
        super().__init__(dict(cfg, layers=layers), w)

    def run(self, tokens):
        x = first = self.w["embed"][np.asarray(tokens)]
        for r, again in enumerate(self.again):
            x = self.one(r, x + first if again else x, self.pos)
        self.pos += len(x)
        return nifunex_ref.norm_about_zero(x, self.w["final.norm"], self.cfg["norm"]["eps"]) @ self.w["head"].T

    def one(self, r, x, pos):
        eps, w, ly, pre = self.cfg["norm"]["eps"], self.w, self.cfg["layers"][r], "l%d." % r
        mx, h = ly["mixer"], nifunex_ref.norm_about_zero(x, w[pre + "norm1"], eps)
        if ly["type"] == "gla":
            y = nifunex_ref.gla(mx, w, pre + "mix.", h, self.s[r], eps)
        else:
            j = r if mx.get("kv_from") is None else mx["kv_from"]
            if j == r:
                c, k = nifunex_ref.latent_rows(mx, w, pre + "mix.", h, pos, eps)
                self.c[r], self.k[r] = np.concatenate([self.c[r], c]), np.concatenate([self.k[r], k])
            y = nifunex_ref.latent_attention(mx, w, pre + "mix.", h, pos, self.c[j], self.k[j])
        x = x + nifunex_ref.norm_about_zero(y, w[pre + "norm1b"], eps)
        if ly.get("mlp"):
            y = nifunex_ref.feed_forward(w, pre + "mlp.", nifunex_ref.norm_about_zero(x, w[pre + "norm2"], eps), ly["mlp"]["limit"])
            x = x + nifunex_ref.norm_about_zero(y, w[pre + "norm2b"], eps)
        return x


@BOTH
def test_loop_of_other_layers(dtype):
    """The loop around recurrent and latent layers with norms behind their sublayers: states and rows per pass, rows of an
    earlier layer read from the same pass."""
    from flexllm_amd import nifunex
    from flexllm_amd.hybrid import HybridModel, group_weights, upload
    cfg = nc.config([nc.gla(mlp=nc.dense()), nc.latent(), nc.latent(heads=2, dim=8, vdim=16, window=50, scale=0.4, kv_from=1, mlp=nc.dense(40)), nc.gla(heads=1)])
    loop = (0, 3, 2)
    w, toks = nc.weights(cfg, 20), nc.tokens(cfg, 60)
    want = LoopedNifunex(cfg, w, loop).run(toks)
    dev = upload(w, list(w))
    layers = [nifunex.layer_descriptor(i, ly, lambda n: w[n].shape) for i, ly in enumerate(cfg["layers"])]
    m = HybridModel(cfg["width"], cfg["vocab"], cfg["norm"]["eps"], layers, group_weights(cfg, dev.__getitem__, dev), dtype=dtype, max_pos=64, norm_add=1.0,
                    post_norms=True, loop=loop)
    for cuts in ([60], [40, 1], [30, 3]):
        close(run(m, toks, cuts), want, dtype, str(cuts))
    m.close()


@BOTH
@pytest.mark.parametrize("m,k,n,split,glu", [(1024, 64, 16384, 16384, 2), (1000, 192, 3648, 3072, 0), (300, 64, 272, 256, 0), (9, 64, 37, 22, 2), (64, 256, 2048, 0, 0)])
def test_gemm_bias_and_gelu_unit(m, k, n, split, glu, dtype):
    from flexllm_amd import ops, to_device
    from flexllm_amd.loader import from_bf16, to_bf16
    r = np.random.default_rng(m + n)
    a, w = [lc.round_bf16(r.standard_normal(s)) for s in ((m, k), (n, k))]
    bias = (r.standard_normal(n) * np.sqrt(k)).astype(np.float32)
    dev = to_device if dtype == "float32" else lambda x: to_device(to_bf16(x))
    y, y32 = ops.linear_float(dev(a), dev(w), split, glu, bias=to_device(bias))
    want = a.astype(np.float64) @ w.astype(np.float64).T + bias
    if split:
        first = lopazen_ref.gelu(want[:, 0:split:2]) * want[:, 1:split:2] if glu else want[:, :split]
        got = y.numpy() if dtype == "float32" else from_bf16(y.numpy())
        tol = 1e-5 if dtype == "float32" else 5e-3
        assert np.all(np.abs(got - first) <= tol * (np.abs(first) + np.sqrt(k)))
    if split < n:
        assert np.all(np.abs(y32.numpy() - want[:, split:]) <= 1e-5 * (np.abs(want[:, split:]) + np.sqrt(k)))


@BOTH
def test_greedy_generation(dtype):
    """generate() follows the oracle's arg-max; near-ties excepted, since one would send the two apart."""
    cfg = lc.mixed()
    w = lc.weights(cfg, 21)
    m = model(cfg, w, dtype)
    prompt = lc.tokens(cfg, 30)
    got = m.generate(prompt, 40)
    assert got == m.generate(prompt, 40, use_graph=False)      # replays against separate launches
    assert got == m.generate(prompt, 40)
    ref = lopazen_ref.Reference(cfg, w)
    logits = ref.run(prompt)[-1]
    for t in got:
        gap = logits.max() - logits[t]
        assert gap <= (1e-3 if dtype == "float32" else 0.15) * logits.std(), gap
        logits = ref.run([t])[-1]
    m.close()


def test_sampled_generation():
    """Top-k draws with given uniform numbers against the oracle's distribution."""
    cfg = lc.mixed(embed_scale=0.4)
    w = lc.weights(cfg, 22)
    w["final.norm"] = lc.round_bf16(w["final.norm"] * 0.25)    # logits close enough together that several tokens are drawn
    m = model(cfg, w, "float32")
    prompt, rands = lc.tokens(cfg, 12), np.random.default_rng(5).random(24).astype(np.float32)
    got = m.generate(prompt, 24, top_k=5, rands=rands)
    assert got == m.generate(prompt, 24, top_k=5, rands=rands, use_graph=False)
    assert len(set(got)) > 3
    ref = lopazen_ref.Reference(cfg, w)
    logits = ref.run(prompt)[-1]
    for t, r in zip(got, rands):
        pick = np.argsort(-logits, kind="stable")[:5]
        e = np.exp(logits[pick] - logits[pick[0]])
        cdf = np.cumsum(e / e.sum())
        k = list(pick).index(t)
        assert (cdf[k - 1] if k else 0.0) - 1e-3 <= r <= cdf[k] + 1e-3
        logits = ref.run([t])[-1]
    m.close()


def test_decoding_continues_a_sequence():
    """step -> decode -> step on one slot: the loop leaves rows and length as single steps would."""
    from flexllm_amd import DeviceArray, to_device
    cfg = lc.mixed()
    w = lc.weights(cfg, 23)
    m = model(cfg, w, "float32")
    prompt = lc.tokens(cfg, 20)
    slot = m.pool.acquire(0)
    m.step(slot, prompt[:-1])
    io, out = to_device(np.array(prompt[-1:], np.int32)), DeviceArray((6,), np.int32)
    m.decode(slot, io, 6, out)
    m.stream().sync()
    gen = out.numpy().tolist()
    assert m.length(slot) == 25 and io.numpy()[0] == gen[-1]
    got = m.step(slot, gen[-1:], [0])
    close(got, expect(cfg, w, prompt + gen)[-1:], "float32")
    m.close()


def test_refusals():
    from flexllm_amd._lib import FlexLLMError
    for cfg, text in ((lc.config([lc.layer(heads=3, kv_heads=2)]), "3 heads on 2"), (lc.config([lc.layer(heads=2, dim=520)]), "at most 512"),
                      (lc.config([lc.layer(every=0)]), "temp_every=0")):
        with pytest.raises(FlexLLMError, match=text):
            model(cfg, lc.weights(cfg, 1), "bfloat16")
    cfg = lc.config([lc.layer()])
    m = model(cfg, lc.weights(cfg, 24), "bfloat16", max_pos=10)
    slot = m.pool.acquire("x")
    with pytest.raises(FlexLLMError, match="max_pos"):
        m.step(slot, [1] * 11)
    m.step(slot, [1] * 10)
    with pytest.raises(FlexLLMError, match="max_pos"):
        m.step(slot, [1])
    m.close()


def test_command_line_and_trace(tmp_path):
    """A model folder through the generation command and through the trace runner."""
    from flexllm_amd import loader
    cfg = lc.mixed()
    w = lc.weights(cfg, 25)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    loader.write_safetensors(str(tmp_path / "model.safetensors"), {n: loader.to_bf16(a) for n, a in w.items()})
    prompt = lc.tokens(cfg, 21)
    m = model(cfg, w, "bfloat16", max_pos=64)
    gen = m.generate(prompt, 9)
    m.close()
    env = dict(os.environ, PYTHONPATH=ROOT)
    p = subprocess.run([sys.executable, "-m", "flexllm_amd.generate", "--model", str(tmp_path), "--prompt", ",".join(map(str, prompt)), "--steps", "9",
                        "--max-pos", "64"], env=env, capture_output=True, text=True, timeout=100)
    assert p.returncode == 0, p.stderr
    assert [int(t) for t in p.stdout.split(",")] == gen
    a, b = lc.tokens(cfg, 30, 2), lc.tokens(cfg, 12, 3)
    steps = [dict(step=0, entries=[dict(id="a", tokens=a[:20], want=[19, 0, 7])], end=[]), dict(step=1, entries=[dict(id="a", tokens=a[20:21], want=[])], end=[]),
             dict(step=2, entries=[dict(id="a", tokens=a[21:], want=[8])], end=["a"]), dict(step=3, entries=[dict(id="b", tokens=b, want=[11])], end=["b"])]
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "30"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert p.returncode == 0, p.stderr
    assert p.stdout.split("\n")[:4] == ["done %d" % i for i in range(4)]
    ra, rb = expect(cfg, w, a), expect(cfg, w, b)
    read = lambda i: np.fromfile(str(tmp_path / ("%d.f32" % i)), "<f4").reshape(-1, cfg["vocab"])
    close(read(0), ra[[19, 0, 7]], "float32")
    close(read(2), ra[[29]], "float32")
    close(read(3), rb[[11]], "float32")
    assert not (tmp_path / "1.f32").exists()
