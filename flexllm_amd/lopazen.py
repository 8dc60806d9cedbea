"""Lopazen: a decoder of grouped-query attention layers whose values are the projected keys (queries and keys normed per head,
a query temperature that grows with the position instead of a rotation, a sink in the softmax), each with a gelu-gated
feed-forward or none; a stretch of the layers may run several times.  Reads config.json and the tensor names of a
checkpoint; the layers themselves are hybrid.HybridModel's."""
import math

from . import synth
from .hybrid import (ConfigError, HybridModel, check_shapes, dense_shapes, group_weights, upload, MIX_SHARED_KV, FF_NONE, FF_DENSE, GLU_GELU)
from .registry import register


def layer_descriptor(i, layer):
    """HybridLayer fields of config layer i."""
    if layer["type"] != "attention":
        raise ConfigError("layer %d: unknown mixer %r" % (i, layer["type"]))
    mx, mlp = layer["mixer"], layer.get("mlp")
    if mx["vdim"] != mx["dim"]:
        raise ConfigError("layer %d: the values are the keys, but vdim %d differs from dim %d" % (i, mx["vdim"], mx["dim"]))
    d = dict(mixer=MIX_SHARED_KV, heads=mx["heads"], kv_heads=mx["kv_heads"], dim=mx["dim"], vdim=mx["vdim"], scale=float(mx["scale"]), sink=1)
    temp = mx.get("q_temp")
    if temp:
        d.update(temp_coef=float(temp["coef"]), temp_every=int(temp["every"]))
    if not mlp:
        d.update(ff_kind=FF_NONE)
    elif mlp["kind"] == "dense":
        d.update(ff_kind=FF_DENSE, ff=mlp["ff"], glu=GLU_GELU)
    else:
        raise ConfigError("layer %d: unknown feed-forward %r" % (i, mlp["kind"]))
    return d


def loop_of(cfg):
    """(start, stop, times) of the repeated layers."""
    lp = cfg.get("loop")
    if not lp:
        return 0, 0, 1
    start, stop, times = int(lp["start"]), int(lp["stop"]), int(lp["times"])
    if not (0 <= start <= stop <= len(cfg["layers"])) or times < 1:
        raise ConfigError("layers %d .. %d of %d cannot run %d times" % (start, stop, len(cfg["layers"]), times))
    return start, stop, times


def tensor_shapes(cfg):
    """{tensor name: shape} of a checkpoint of this configuration."""
    W = cfg["width"]
    out = {"embed": (cfg["vocab"], W), "final.norm": (W,)}
    for i, ly in enumerate(cfg["layers"]):
        mx, mlp, pre = ly["mixer"], ly.get("mlp"), "l%d." % i
        for n in ("norm1",) + (("norm2",) if mlp else ()):
            out[pre + n] = (W,)
        m, HD, GD = pre + "mix.", mx["heads"] * mx["dim"], mx["kv_heads"] * mx["dim"]
        out.update({m + "q": (HD, W), m + "q.b": (HD,), m + "k": (GD, W), m + "k.b": (GD,), m + "q.norm": (mx["dim"],), m + "k.norm": (mx["dim"],),
                    m + "o": (W, mx["heads"] * mx["vdim"])})
        if mlp:
            dense_shapes(out, pre + "mlp.", mlp["ff"], W)
    return out


@register("Lopazen")
class Lopazen(HybridModel):
    def __init__(self, cfg, weights, dtype="bfloat16", max_pos=4096, slots=1):
        """weights: group_weights' structure."""
        self.cfg = cfg
        layers = [layer_descriptor(i, ly) for i, ly in enumerate(cfg["layers"])]
        super().__init__(cfg["width"], cfg["vocab"], cfg["norm"]["eps"], layers, weights, dtype=dtype, max_pos=max_pos, slots=slots,
                         embed_scale=cfg["embedding"]["scale"], loop=loop_of(cfg))

    @classmethod
    def from_tensors(cls, cfg, tensors, **kw):
        """tensors: {name: host array}, bfloat16 as uint16 bit patterns or any float array (rounded to bfloat16)."""
        want = tensor_shapes(cfg)
        check_shapes(tensors, want)
        dev = upload(tensors, want)
        return cls(cfg, group_weights(cfg, dev.__getitem__, dev), **kw)

    @classmethod
    def synthetic(cls, cfg, seed=1, **kw):
        """Random weights filled on the device: projections uniform with unit-variance outputs, norms near their identity."""
        dev = {}
        for t, (name, shape) in enumerate(sorted(tensor_shapes(cfg).items())):
            r = math.sqrt(3.0 / shape[-1])
            lo, hi = (-r, r) if len(shape) == 2 else (0.9, 1.1)
            if name.endswith(".b"):
                lo, hi = -0.2, 0.2
            elif name == "embed":
                lo, hi = -r, r
            dev[name] = synth.device_uniform_bf16(shape, seed * 1000003 + t, lo, hi)
        return cls(cfg, group_weights(cfg, dev.__getitem__, dev), **kw)
