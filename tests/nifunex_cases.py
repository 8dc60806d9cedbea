"""Small random Nifunex configurations and weights for the tests."""
import numpy as np

from flexllm_amd import loader, nifunex


def latent(heads=3, dim=24, rot_dim=16, vdim=40, kv_rank=48, window=33, scale=0.2, kv_from=None, base=10000.0,
           scaling=dict(factor=4.0, original=64, fast=8.0, slow=1.0), mlp=None):
    mx = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, scale=scale, rot=dict(base=base, dims=rot_dim))
    if scaling:
        mx["rot"]["scaling"] = dict(scaling)
    if window:
        mx["mask"] = dict(size=window)
    if kv_from is not None:
        mx["kv_from"] = kv_from
    return dict(type="latent_attention", mixer=mx, mlp=mlp)


def gla(heads=2, dim=20, vdim=36, tau=8.0, mlp=None):
    return dict(type="gla", mixer=dict(heads=heads, dim=dim, vdim=vdim, tau=tau), mlp=mlp)


def dense(ff=88, limit=1.25):
    return dict(kind="dense", ff=ff, limit=limit)


def moe(experts=6, top=2, ff=40, limit=0.75, shared=56, shared_limit=2.0):
    m = dict(kind="moe", router=dict(experts=experts, top=top), expert=dict(ff=ff, limit=limit))
    if shared:
        m["shared"] = dict(ff=shared, limit=shared_limit)
    return m


def config(layers, width=160, vocab=300, eps=1e-5):
    return dict(architecture="Nifunex", width=width, vocab=vocab, norm=dict(eps=eps), layers=layers)


def mixed(**kw):
    """Every mechanism once, no two sizes alike."""
    return config([gla(mlp=dense()), latent(mlp=moe()), latent(heads=5, dim=16, vdim=24, window=9, scale=0.3, kv_from=1, mlp=moe(5, 3, 24, 1.5, 0)),
                   gla(heads=3, dim=36, vdim=20, tau=2.0), latent(heads=2, kv_rank=72, rot_dim=8, window=70, scaling=None, base=500.0, mlp=dense(72, 2.0))], **kw)


def weights(cfg, seed=0, a_rank=12):
    """{name: float32 array with bfloat16 values}; sized so that every sublayer and every gate is alive."""
    r = np.random.default_rng(seed)
    out = {}
    for name, shape in nifunex.tensor_shapes(cfg, a_rank).items():
        if name.endswith(("norm1", "norm2", "norm1b", "norm2b", "final.norm")):
            a = r.uniform(-0.4, 0.4, shape)
        elif name.endswith(("dkv.norm", "mix.norm")):
            a = r.uniform(0.6, 1.4, shape)
        elif name.endswith("a2.b"):
            a = r.uniform(-1.0, 5.0, shape)
        elif name == "embed":
            a = r.standard_normal(shape)
        elif name.endswith("router"):
            a = r.standard_normal(shape) * 2.0 / np.sqrt(shape[-1])
        else:
            a = r.standard_normal(shape) * 1.2 / np.sqrt(shape[-1])
        out[name] = loader.from_bf16(loader.to_bf16(a.astype(np.float32)))
    return out


def tokens(cfg, n, seed=1):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()


def rel_err(got, want):
    """Error of each row of logits, mean taken off, in units of the rows' overall spread."""
    d = got - want
    d = d - d.mean(-1, keepdims=True)
    w = want - want.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / np.sqrt((w * w).mean())


LIMIT = {"float32": 1e-4, "bfloat16": 6e-2}
