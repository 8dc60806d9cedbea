"""Small random Lopazen configurations and weights for the tests."""
import numpy as np

from flexllm_amd import loader, lopazen
from nifunex_cases import LIMIT, rel_err, tokens  # noqa: F401


def dense(ff=88):
    return dict(kind="dense", ff=ff)


def layer(heads=6, kv_heads=2, dim=24, scale=0.2, coef=0.4, every=16, mlp=None):
    return dict(type="attention", mlp=mlp, mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=scale, q_temp=dict(coef=coef, every=every)))


def config(layers, loop=(0, 0, 1), width=160, vocab=300, eps=1e-5, embed_scale=3.0):
    return dict(architecture="Lopazen", width=width, vocab=vocab, norm=dict(eps=eps), embedding=dict(scale=embed_scale), layers=layers,
                loop=dict(zip(("start", "stop", "times"), loop)))


def mixed(**kw):
    """Every branch once, no two sizes alike."""
    return config([layer(mlp=dense()), layer(heads=4, kv_heads=4, dim=40, scale=0.3, coef=0.7, every=9, mlp=dense(60)),
                   layer(heads=5, kv_heads=1, dim=16, scale=0.25, coef=-0.2, every=33), layer(heads=8, kv_heads=2, dim=64, scale=0.1, every=50, mlp=dense(131))],
                  loop=(1, 3, 3), **kw)


def weights(cfg, seed=0):
    """{name: float32 array with bfloat16 values}; sized so that every sublayer is alive and residuals stay of one size."""
    r = np.random.default_rng(seed)
    out = {}
    for name, shape in lopazen.tensor_shapes(cfg).items():
        if "norm" in name:
            a = r.uniform(0.6, 1.4, shape)
        elif name.endswith(".b"):
            a = r.uniform(-0.6, 0.6, shape)
        elif name == "embed":
            a = r.standard_normal(shape) * 0.3
        else:
            a = r.standard_normal(shape) * 1.1 / np.sqrt(shape[-1])
        out[name] = round_bf16(a)
    return out


def round_bf16(a):
    return loader.from_bf16(loader.to_bf16(np.asarray(a, np.float32)))


def split_qk(cfg, w, i=0):
    """(query, key, value) [vocab][heads or kv heads][dim] that the tokens of a one-layer model have ahead of temperature and
    scale."""
    from oracle import lopazen_ref as ref
    mx, eps = cfg["layers"][i]["mixer"], cfg["norm"]["eps"]
    h = ref.rms_norm(w["embed"].astype(np.float64) * cfg["embedding"]["scale"], w["l%d.norm1" % i], eps)
    m = "l%d.mix." % i
    q = (h @ w[m + "q"].T + w[m + "q.b"]).reshape(len(h), mx["heads"], mx["dim"])
    k, v = ref.key_values(mx, w, m, h, eps)
    return ref.rms_norm(q, w[m + "q.norm"], eps), k, v
