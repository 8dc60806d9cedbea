"""Nifunex on the GPU against the plain statement of its equations (oracle/nifunex_ref.py): each mechanism alone, sizes of
many kinds, prompts against decoding and portions, slots used again, edges of windows, long decoding, generation."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import nifunex_cases as nc
from oracle import nifunex_ref

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
BOTH = pytest.mark.parametrize("dtype", ["float32", "bfloat16"])


def model(cfg, w, dtype, max_pos=512, slots=1):
    from flexllm_amd.nifunex import Nifunex
    return Nifunex.from_tensors(cfg, w, dtype=dtype, max_pos=max_pos, slots=slots)


def run(m, toks, cuts, slot=None):
    """Logits of every token, fed in portions of the given sizes (the last one repeats)."""
    key = object()
    s = m.pool.acquire(key) if slot is None else slot
    out, p, i = [], 0, 0
    while p < len(toks):
        c = min(cuts[min(i, len(cuts) - 1)], len(toks) - p)
        out.append(m.step(s, toks[p:p + c], range(c)))
        p += c
        i += 1
    m.check()
    if slot is None:
        m.pool.release(key)
    return np.concatenate(out)


def expect(cfg, w, toks):
    return nifunex_ref.Reference(cfg, w).run(toks)


def close(got, want, dtype, what=""):
    e = nc.rel_err(got, want)
    assert np.isfinite(got).all(), what
    if dtype == "bfloat16" and len(e) > 20:
        # rounding may decide a router's close call differently: a few places may differ by an expert
        e = np.sort(e)[:int(0.95 * len(e))]
    assert e.max() < nc.LIMIT[dtype], "%s: error %.3g at place %d (mean %.3g)" % (what, e.max(), e.argmax(), e.mean())


ALONE = {
    "gla": nc.config([nc.gla()]),
    "gla one head, wide values": nc.config([nc.gla(heads=1, dim=16, vdim=96, tau=1.0)]),
    "gla beyond one chunk size": nc.config([nc.gla(heads=2, dim=144, vdim=136)]),
    "gla beyond the chunk kernels": nc.config([nc.gla(heads=1, dim=264, vdim=24)]),
    "gla, 72 channels": nc.config([nc.gla(heads=2, dim=72, vdim=128)]),
    "gla, 128 channels": nc.config([nc.gla(heads=1, dim=128, vdim=88, tau=16.0)]),
    "latent": nc.config([nc.latent()]),
    "latent without window": nc.config([nc.latent(window=None)]),
    "latent without yarn": nc.config([nc.latent(scaling=None)]),
    "latent, window of one": nc.config([nc.latent(window=1)]),
    "latent, window of two": nc.config([nc.latent(window=2)]),
    "latent, large heads": nc.config([nc.latent(heads=2, dim=128, rot_dim=64, vdim=128, kv_rank=200, window=100, scale=0.07)]),
    "latent, wide values": nc.config([nc.latent(heads=1, dim=64, rot_dim=32, vdim=160, kv_rank=96)]),
    "latent, odd sizes": nc.config([nc.latent(heads=3, dim=10, rot_dim=6, vdim=7, kv_rank=30)]),
    "latent, other layer's rows": nc.config([nc.latent(window=20), nc.latent(heads=2, dim=8, vdim=16, window=50, scale=0.4, kv_from=0)]),
    "latent, long rows": nc.config([nc.latent(heads=1, dim=16, vdim=16, kv_rank=2100)]),
    "dense, vectors of some length": nc.config([nc.gla(mlp=nc.dense(ff=3000))], width=64),
    "dense, long vectors": nc.config([nc.gla(mlp=nc.dense(ff=8300))], width=64),
    "dense": nc.config([nc.gla(mlp=nc.dense(ff=100, limit=0.5))]),
    "mixture": nc.config([nc.gla(mlp=nc.moe(shared=0))]),
    "mixture, top 1": nc.config([nc.gla(mlp=nc.moe(experts=9, top=1, shared=0))]),
    "mixture, all experts": nc.config([nc.gla(mlp=nc.moe(experts=4, top=4, ff=30))]),
    "mixture, more than 64 experts": nc.config([nc.gla(mlp=nc.moe(experts=70, top=5, ff=16))]),
    "mixture with shared expert": nc.config([nc.latent(mlp=nc.moe(shared=64))]),
    "odd width and vocabulary": nc.config([nc.gla(mlp=nc.dense(ff=33)), nc.latent(mlp=nc.moe(shared=27))], width=90, vocab=131),
    "everything": nc.mixed(),
}


@BOTH
@pytest.mark.parametrize("name", list(ALONE))
def test_mechanism(name, dtype):
    cfg = ALONE[name]
    w = nc.weights(cfg, 3)
    toks = nc.tokens(cfg, 90)
    want = expect(cfg, w, toks)
    m = model(cfg, w, dtype)
    close(run(m, toks, [90]), want, dtype, "whole prompt")
    close(run(m, toks, [70, 1]), want, dtype, "decoded")
    m.close()


@BOTH
def test_residual_after_every_layer(dtype):
    cfg = nc.mixed()
    w, toks = nc.weights(cfg, 4), nc.tokens(cfg, 40)
    trace = []
    nifunex_ref.Reference(cfg, w).run(toks, trace)
    m = model(cfg, w, dtype)
    for n in (40, 5):                                      # both schedules
        slot = m.pool.acquire(n)
        _, got = m.step(slot, toks[:n], [n - 1], layers=True)
        m.pool.release(n)
        for i, ref in enumerate(trace):
            err = np.abs(got[i] - ref[:n]).max() / np.sqrt((ref ** 2).mean())
            assert err < (2e-5 if dtype == "float32" else 8e-2), "layer %d, %d tokens: %.3g" % (i, n, err)
    m.close()


@BOTH
@pytest.mark.parametrize("cuts", [[1], [2], [3, 2], [7, 9, 8], [16], [17, 1, 64], [63, 65, 2], [64], [129, 2]])
def test_portions(cuts, dtype):
    cfg = nc.mixed()
    w, toks = nc.weights(cfg, 5), nc.tokens(cfg, 200)
    m = model(cfg, w, dtype)
    close(run(m, toks, cuts), expect(cfg, w, toks), dtype, str(cuts))
    m.close()


def test_prompt_equals_decoding():
    """The same logits from a prompt in one go and from its tokens one by one, well inside bfloat16's step."""
    cfg = nc.mixed()
    w, toks = nc.weights(cfg, 6), nc.tokens(cfg, 150)
    m = model(cfg, w, "float32")
    close(run(m, toks, [150]), run(m, toks, [1]), "float32")
    m.close()


@BOTH
def test_long_prompt_and_long_decoding(dtype):
    cfg = nc.config([nc.gla(dim=32, vdim=32, tau=16.0, mlp=nc.dense()), nc.latent(heads=2, dim=32, rot_dim=32, vdim=32, kv_rank=64, window=300, mlp=nc.moe())])
    w, toks = nc.weights(cfg, 7), nc.tokens(cfg, 900)
    want = expect(cfg, w, toks)
    m = model(cfg, w, dtype, max_pos=900)
    close(run(m, toks, [900]), want, dtype, "prompt of 900")
    close(run(m, toks, [500, 1]), want, dtype, "400 decoded tokens")
    m.close()


@BOTH
def test_strong_and_weak_decays(dtype):
    """Channels that forget within a token beside channels that keep everything."""
    cfg = nc.config([nc.gla(heads=2, dim=32, vdim=24, tau=1.0), nc.gla(heads=2, dim=32, vdim=24, tau=16.0)])
    w = nc.weights(cfg, 8)
    b = w["l0.mix.a2.b"]
    b[:] = np.where(np.arange(b.size) % 3 == 0, -60.0, np.where(np.arange(b.size) % 3 == 1, 30.0, 0.0))
    toks = nc.tokens(cfg, 200)
    m = model(cfg, w, dtype)
    for cuts in ([200], [130, 1]):
        close(run(m, toks, cuts), expect(cfg, w, toks), dtype, str(cuts))
    m.close()


@BOTH
def test_state_reaches_far_back(dtype):
    """One token writes what a much later one reads, through the state alone."""
    cfg = nc.config([nc.gla(heads=1, dim=16, vdim=32, tau=16.0)], vocab=64)
    w = nc.weights(cfg, 9)
    w["l0.mix.a2.b"][:] = 24.0                             # hardly any decay
    w["l0.mix.a2"][:] = 0.0
    # the keys of all tokens but one lie in half of the channels, the last token's query in the other half
    h = nifunex_ref.norm_about_zero(w["embed"], w["l0.norm1"], 1e-5)
    far, asks = 5, 6
    keys = np.zeros((64, 16), np.float32)
    keys[:, :8], keys[:, 8:] = 0.05, 0.2
    keys[far, :8], keys[far, 8:] = 0.0, 8.0
    queries = np.zeros((64, 16), np.float32)
    queries[:, :8] = 1.0
    queries[asks, :8], queries[asks, 8:] = 0.0, 2.0
    inv = np.linalg.pinv(h)
    from flexllm_amd.loader import from_bf16, to_bf16
    w["l0.mix.k"], w["l0.mix.q"] = [from_bf16(to_bf16((inv @ a).T.astype(np.float32))) for a in (keys, queries)]
    fill = [t for t in nc.tokens(cfg, 400) if t not in (far, asks)]
    toks, other = [far] + fill[:300] + [asks], [fill[301]] + fill[:300] + [asks]
    want, want2 = expect(cfg, w, toks), expect(cfg, w, other)
    assert nc.rel_err(want[-1:], want2[-1:])[0] > 0.3      # the case is sharp
    m = model(cfg, w, dtype)
    for cuts in ([302], [200, 1], [64]):
        close(run(m, toks, cuts)[-1:], want[-1:], dtype, str(cuts))
        close(run(m, other, cuts)[-1:], want2[-1:], dtype, str(cuts))
    m.close()


@BOTH
@pytest.mark.parametrize("window", [5, 64, 65, 128, 150])
def test_window_edge(window, dtype):
    """A key whose score stands out, just inside and just outside the window, in a prompt and in decoding, with the query
    at various places relative to tile and split borders."""
    cfg = nc.config([nc.latent(heads=1, dim=32, rot_dim=8, vdim=32, kv_rank=48, window=window, scale=1.0, scaling=None)], vocab=60)
    w = nc.weights(cfg, 10)
    w["l0.mix.dkv"][48:] = 0.0                             # no rotated part: scores do not depend on places
    h = nifunex_ref.norm_about_zero(w["embed"], w["l0.norm1"], 1e-5)
    q = (h @ w["l0.mix.q"].T)[:, :32]
    k = nifunex_ref.rms(h @ w["l0.mix.dkv"][:48].T, 1e-5) * w["l0.mix.dkv.norm"] @ w["l0.mix.uk"].T
    s = q @ k.T
    asks, key = np.unravel_index(np.argmax(s - np.median(s, 1, keepdims=True)), s.shape)
    fill = [t for t in np.argsort(s[asks])[:20] if t not in (asks, key)]
    m = model(cfg, w, dtype)
    rng = np.random.default_rng(0)
    for n in (window, window + 1, 190, 192, 193):
        outs = []
        for dist in (window - 1, window):
            if dist > n:
                continue
            toks = rng.choice(fill, n + 1).tolist()
            toks[n], toks[n - dist] = int(asks), int(key)
            want = expect(cfg, w, toks)
            for cuts in ([n + 1], [n, 1], [max(n - 3, 1), 2]):
                close(run(m, toks, cuts)[-1:], want[-1:], dtype, "n=%d distance=%d cuts=%s" % (n, dist, cuts))
            outs.append(want[-1])
        if len(outs) == 2:
            assert nc.rel_err(outs[0][None], outs[1][None])[0] > 0.2
    m.close()


@BOTH
def test_slots(dtype):
    """Sequences in several slots, interleaved, and a slot that is used again, equal a sequence alone."""
    cfg = nc.mixed()
    w = nc.weights(cfg, 11)
    m = model(cfg, w, dtype, slots=2)
    a, b, c = nc.tokens(cfg, 120, 1), nc.tokens(cfg, 61, 2), nc.tokens(cfg, 40, 3)
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


@BOTH
def test_many_visible_keys(dtype):
    """More keys than one tile per split holds, so that the splits' running maxima come into play."""
    cfg = nc.config([nc.latent(heads=1, dim=16, rot_dim=8, vdim=16, kv_rank=512, window=None, scale=0.5)], width=96, vocab=90)
    w, toks = nc.weights(cfg, 19), nc.tokens(cfg, 2310)
    want = expect(cfg, w, toks)
    m = model(cfg, w, dtype, max_pos=2600)
    slot = m.pool.acquire(0)
    m.step(slot, toks[:2300])
    got = [m.step(slot, toks[2300 + i:2301 + i], [0]) for i in range(10)]
    close(np.concatenate(got), want[2300:], dtype)
    m.close()


@BOTH
@pytest.mark.parametrize("m,k,n,split,glu", [(1024, 64, 16384, 16384, 1), (1024, 128, 4096, 4096, 0), (1000, 192, 3648, 3072, 0), (300, 64, 272, 256, 0),
                                             (64, 256, 2048, 0, 0), (9, 64, 37, 22, 1), (130, 64, 301, 150, 0), (2048, 64, 2112, 2048, 1)])
def test_gemm(m, k, n, split, glu, dtype):
    """Every tile shape of the GEMM, ragged sizes, the split between the two outputs, the gated unit in the epilogue."""
    from flexllm_amd import ops, to_device
    from flexllm_amd.loader import from_bf16, to_bf16
    r = np.random.default_rng(m + n)
    a, w = [from_bf16(to_bf16(r.standard_normal(s).astype(np.float32))) for s in ((m, k), (n, k))]
    dev = to_device if dtype == "float32" else lambda x: to_device(to_bf16(x))
    y, y32 = ops.linear_float(dev(a), dev(w), split, bool(glu), 3.0)
    want = a.astype(np.float64) @ w.astype(np.float64).T
    if split:
        first = nifunex_ref.clamped_glu(want[:, 0:split:2], want[:, 1:split:2], 3.0) if glu else want[:, :split]
        got = y.numpy() if dtype == "float32" else from_bf16(y.numpy())
        tol = 1e-5 if dtype == "float32" else 5e-3
        assert np.all(np.abs(got - first) <= tol * (np.abs(first) + np.sqrt(k)))
    if split < n:
        assert np.all(np.abs(y32.numpy() - want[:, split:]) <= 1e-5 * (np.abs(want[:, split:]) + np.sqrt(k)))


def test_first_tokens():
    cfg = nc.mixed()
    w = nc.weights(cfg, 12)
    m = model(cfg, w, "float32")
    for n in (1, 2, 3, 8, 9):
        toks = nc.tokens(cfg, n, n)
        close(run(m, toks, [n]), expect(cfg, w, toks), "float32", "%d tokens" % n)
    m.close()


def test_many_pieces():
    """More tokens in one call than the library takes at a time."""
    cfg = nc.config([nc.gla(dim=16, vdim=16), nc.latent(heads=1, dim=16, rot_dim=8, vdim=16, kv_rank=16, window=12)], width=64, vocab=80)
    w, toks = nc.weights(cfg, 13), nc.tokens(cfg, 4200)
    want = expect(cfg, w, toks)
    m = model(cfg, w, "float32", max_pos=4200)
    slot = m.pool.acquire(0)
    places = [0, 4094, 4095, 4096, 4097, 4199]
    close(m.step(slot, toks, places), want[places], "float32")
    m.close()


@BOTH
def test_greedy_generation(dtype):
    """generate() follows the oracle's arg-max; near-ties excepted, since one would send the two apart."""
    cfg = nc.mixed()
    w = nc.weights(cfg, 14)
    m = model(cfg, w, dtype)
    prompt = nc.tokens(cfg, 30)
    got = m.generate(prompt, 40)
    assert got == m.generate(prompt, 40, use_graph=False)      # replays against separate launches
    assert got == m.generate(prompt, 40)
    ref = nifunex_ref.Reference(cfg, w)
    logits = ref.run(prompt)[-1]
    for t in got:
        gap = logits.max() - logits[t]
        assert gap <= (1e-3 if dtype == "float32" else 0.15) * logits.std(), gap
        logits = ref.run([t])[-1]
    m.close()


def test_sampled_generation():
    """Top-k draws with given uniform numbers against the oracle's distribution."""
    cfg = nc.mixed()
    w = nc.weights(cfg, 15)
    m = model(cfg, w, "float32")
    prompt, rands = nc.tokens(cfg, 12), np.random.default_rng(5).random(24).astype(np.float32)
    got = m.generate(prompt, 24, top_k=5, rands=rands)
    assert got == m.generate(prompt, 24, top_k=5, rands=rands, use_graph=False)
    assert len(set(got)) > 3
    ref = nifunex_ref.Reference(cfg, w)
    logits = ref.run(prompt)[-1]
    for t, r in zip(got, rands):
        pick = np.argsort(-logits, kind="stable")[:5]
        e = np.exp(logits[pick] - logits[pick[0]])
        cdf = np.cumsum(e / e.sum())
        k = list(pick).index(t)
        lo, hi = (cdf[k - 1] if k else 0.0), cdf[k]
        assert lo - 1e-3 <= r <= hi + 1e-3
        logits = ref.run([t])[-1]
    m.close()


def test_decoding_continues_a_sequence():
    """step -> decode -> step on one slot: the loop leaves cache, state and length as single steps would."""
    from flexllm_amd import DeviceArray, to_device
    cfg = nc.mixed()
    w = nc.weights(cfg, 16)
    m = model(cfg, w, "float32")
    prompt = nc.tokens(cfg, 20)
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


def test_errors():
    from flexllm_amd._lib import FlexLLMError
    from flexllm_amd.slots import NoFreeSlot
    cfg = nc.config([nc.gla()])
    w = nc.weights(cfg, 17)
    m = model(cfg, w, "bfloat16", max_pos=10)
    slot = m.pool.acquire("x")
    with pytest.raises(NoFreeSlot):
        m.pool.acquire("y")
    with pytest.raises(FlexLLMError, match="max_pos"):
        m.step(slot, [1] * 11)
    m.step(slot, [1] * 10)
    with pytest.raises(FlexLLMError, match="max_pos"):
        m.step(slot, [1])
    m.pool.release("x")
    slot = m.pool.acquire("y")
    with pytest.raises(FlexLLMError, match="ascending"):
        m.step(slot, [1, 2], [1, 0])
    m.step(slot, [cfg["vocab"]])
    with pytest.raises(FlexLLMError, match="outside the vocabulary"):
        m.check()
    m.check()
    m.close()


def test_command_line_and_trace(tmp_path):
    """A model folder through the generation command and through the trace runner."""
    from flexllm_amd import loader
    cfg = nc.mixed()
    w = nc.weights(cfg, 18)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    loader.write_safetensors(str(tmp_path / "model.safetensors"), {n: loader.to_bf16(a) for n, a in w.items()})
    prompt = nc.tokens(cfg, 21)
    m = model(cfg, w, "bfloat16")
    gen = m.generate(prompt, 9)
    m.close()
    env = dict(os.environ, PYTHONPATH=ROOT)
    p = subprocess.run([sys.executable, "-m", "flexllm_amd.generate", "--model", str(tmp_path), "--prompt", ",".join(map(str, prompt)), "--steps", "9",
                        "--max-pos", "64"], env=env, capture_output=True, text=True, timeout=100)
    assert p.returncode == 0, p.stderr
    assert [int(t) for t in p.stdout.split(",")] == gen
    a, b = nc.tokens(cfg, 30, 2), nc.tokens(cfg, 12, 3)
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
