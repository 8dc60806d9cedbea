"""Nifunex: a decoder whose layers are latent attention (sliding window, YaRN-scaled rotary part, possibly on another
layer's cached rows) or gated linear attention, each with a dense or a mixture feed-forward, norms before and after every
sublayer.  Reads config.json and the tensor names of a checkpoint; the layers themselves are hybrid.HybridModel's."""
import math

from . import loader, synth
from .hybrid import (ConfigError, HybridModel, check_shapes, dense_shapes, group_weights, upload, MIX_LATENT, MIX_GLA, FF_NONE, FF_DENSE, FF_MOE)
from .registry import register


def layer_descriptor(i, layer, shape):
    """HybridLayer fields of config layer i; shape(name) gives a tensor's shape (for what the config leaves to them)."""
    mx, d = layer["mixer"], {}
    d.update(heads=mx["heads"], dim=mx["dim"], vdim=mx["vdim"])
    if layer["type"] == "latent_attention":
        rot = mx["rot"]
        if rot["dims"] != mx["rot_dim"]:
            raise ConfigError("layer %d: rot.dims %d differs from rot_dim %d" % (i, rot["dims"], mx["rot_dim"]))
        kv_from = mx.get("kv_from")
        d.update(mixer=MIX_LATENT, rot_dim=mx["rot_dim"], kv_rank=mx["kv_rank"], window=int((mx.get("mask") or {}).get("size") or 0),
                 kv_from=-1 if kv_from is None else int(kv_from), scale=float(mx["scale"]), rot_base=float(rot["base"]))
        sc = rot.get("scaling")
        if sc:
            d.update(yarn=1, yarn_factor=float(sc["factor"]), yarn_original=float(sc["original"]), yarn_fast=float(sc["fast"]),
                     yarn_slow=float(sc["slow"]))
    elif layer["type"] == "gla":
        d.update(mixer=MIX_GLA, a_rank=int(shape("l%d.mix.a1" % i)[0]), tau=float(mx["tau"]))
    else:
        raise ConfigError("layer %d: unknown mixer %r" % (i, layer["type"]))
    mlp = layer.get("mlp")
    if not mlp:
        d.update(ff_kind=FF_NONE)
    elif mlp["kind"] == "dense":
        d.update(ff_kind=FF_DENSE, ff=mlp["ff"], limit=float(mlp["limit"]))
    elif mlp["kind"] == "moe":
        shared = mlp.get("shared")
        d.update(ff_kind=FF_MOE, ff=mlp["expert"]["ff"], limit=float(mlp["expert"]["limit"]), experts=mlp["router"]["experts"],
                 top=mlp["router"]["top"])
        if shared:
            d.update(shared_ff=shared["ff"], shared_limit=float(shared["limit"]))
    else:
        raise ConfigError("layer %d: unknown feed-forward %r" % (i, mlp["kind"]))
    return d


def tensor_shapes(cfg, a_rank=16):
    """{tensor name: shape} of a checkpoint of this configuration; a_rank: rank of the decay projection, which the
    configuration leaves to the tensors."""
    W, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"]), "final.norm": (cfg["width"],), "head": (cfg["vocab"], cfg["width"])}
    for i, ly in enumerate(cfg["layers"]):
        mx, mlp, pre = ly["mixer"], ly.get("mlp"), "l%d." % i
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if mlp else ()):
            out[pre + n] = (W,)
        m, H = pre + "mix.", mx["heads"]
        HD, HV = H * mx["dim"], H * mx["vdim"]
        if ly["type"] == "gla":
            out.update({m + "q": (HD, W), m + "k": (HD, W), m + "v": (HV, W), m + "g": (HV, W), m + "norm": (mx["vdim"],),
                        m + "a1": (a_rank, W), m + "a2": (HD, a_rank), m + "a2.b": (HD,)})
        else:
            out.update({m + "q": (H * (mx["dim"] + mx["rot_dim"]), W), m + "uk": (HD, mx["kv_rank"]), m + "uv": (HV, mx["kv_rank"])})
            if mx.get("kv_from") is None:
                out.update({m + "dkv": (mx["kv_rank"] + mx["rot_dim"], W), m + "dkv.norm": (mx["kv_rank"],)})
        out[m + "o"] = (W, HV)
        if not mlp:
            continue
        f = pre + "mlp."
        if mlp["kind"] == "dense":
            dense_shapes(out, f, mlp["ff"], W)
        else:
            for e in range(mlp["router"]["experts"]):
                dense_shapes(out, "%se%d." % (f, e), mlp["expert"]["ff"], W)
            out[f + "router"] = (mlp["router"]["experts"], W)
            if mlp.get("shared"):
                dense_shapes(out, f + "shared.", mlp["shared"]["ff"], W)
                out[f + "shared.sg"] = (1, W)
    return out


@register("Nifunex")
class Nifunex(HybridModel):
    def __init__(self, cfg, weights, shapes, dtype="bfloat16", max_pos=4096, slots=1):
        """weights: group_weights' structure; shapes: {tensor name: shape}."""
        self.cfg = cfg
        layers = [layer_descriptor(i, ly, shapes.__getitem__) for i, ly in enumerate(cfg["layers"])]
        super().__init__(cfg["width"], cfg["vocab"], cfg["norm"]["eps"], layers, weights, dtype=dtype, max_pos=max_pos, slots=slots,
                         norm_add=1.0, post_norms=True)

    @classmethod
    def from_tensors(cls, cfg, tensors, **kw):
        """tensors: {name: host array}, bfloat16 as uint16 bit patterns or any float array (rounded to bfloat16)."""
        want = tensor_shapes(cfg)
        check_shapes(tensors, want, lambda name: (0,) if name.endswith(".mix.a1") else (1,) if name.endswith(".mix.a2") else ())
        for i in range(len(cfg["layers"])):
            m = "l%d.mix." % i
            if m + "a1" in want and tensors[m + "a1"].shape[0] != tensors[m + "a2"].shape[1]:
                raise loader.ParameterError("%sa1 and %sa2 disagree about the rank" % (m, m))
        dev = upload(tensors, want)
        return cls(cfg, group_weights(cfg, dev.__getitem__, dev), {n: tuple(t.shape) for n, t in tensors.items()}, **kw)

    @classmethod
    def synthetic(cls, cfg, seed=1, a_rank=16, **kw):
        """Random weights filled on the device: projections uniform with unit-variance outputs, norms near their identity."""
        shapes = tensor_shapes(cfg, a_rank)
        dev = {}
        for t, (name, shape) in enumerate(sorted(shapes.items())):
            r = math.sqrt(3.0 / shape[-1])
            lo, hi = (-r, r) if len(shape) == 2 else (-0.1, 0.1)
            if name.endswith(("dkv.norm", "mix.norm")):
                lo, hi = 0.9, 1.1
            elif name.endswith("a2.b"):
                lo, hi = 1.0, 4.0
            elif name == "embed":
                lo, hi = -1.7, 1.7
            dev[name] = synth.device_uniform_bf16(shape, seed * 1000003 + t, lo, hi)
        return cls(cfg, group_weights(cfg, dev.__getitem__, dev), shapes, **kw)

