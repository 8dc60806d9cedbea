"""Decoder of floating-point layers chosen one by one (latent attention, attention over shared key/value rows, gated linear
attention, dense and mixture feed-forwards): the wrapper over the C ABI model object (flexllm_hybrid_*), shared by every design that is made of these
layers.  A design supplies layer descriptors (fields of _lib.HybridLayer), the shapes of its tensors and what surrounds the
layers."""
import ctypes as C
import os

import numpy as np

from . import loader
from ._lib import lib, check, HybridConfig, HybridLayer, HybridLayerWeights, HybridWeights
from .device import DeviceArray, Stream, to_device, _s
from .slots import SlotPool

MIX_LATENT, MIX_GLA, MIX_SHARED_KV = 0, 1, 2
FF_NONE, FF_DENSE, FF_MOE = 0, 1, 2
GLU_CLAMPED, GLU_GELU = 0, 1
DTYPES = {"bfloat16": 0, "float32": 1}


class ConfigError(ValueError):
    pass


# field of HybridLayerWeights -> tensor name behind 'l<i>.', 'l<i>.mix.', 'l<i>.mlp.'
_NORMS = dict(norm1="norm1", norm1b="norm1b", norm2="norm2", norm2b="norm2b")
_MIX = dict(q="q", o="o", dkv="dkv", dkv_norm="dkv.norm", uk="uk", uv="uv", k="k", v="v", g="g", a1="a1", a2="a2", a2_bias="a2.b", head_norm="norm",
            q_bias="q.b", k_bias="k.b", q_norm="q.norm", k_norm="k.norm")
_MLP = dict(gate="gate", up="up", down="down", router="router", shared_gate="shared.gate", shared_up="shared.up",
            shared_down="shared.down", shared_sg="shared.sg")


def group_weights(cfg, tensor, names):
    """The weights structure of HybridModel; tensor(name) gives a device array, names the tensors that there are.  Without a
    tensor "head" the embedding matrix is the head."""
    embed = tensor("embed")
    out = {"embed": embed, "final_norm": tensor("final.norm"), "head": tensor("head") if "head" in names else embed, "layers": []}
    for i, ly in enumerate(cfg["layers"]):
        w = {}
        for table, pre in ((_NORMS, "l%d." % i), (_MIX, "l%d.mix." % i), (_MLP, "l%d.mlp." % i)):
            w.update({f: tensor(pre + n) for f, n in table.items() if pre + n in names})
        mlp = ly.get("mlp")
        if mlp and mlp["kind"] == "moe":
            for part in ("gate", "up", "down"):
                w["expert_" + part] = [tensor("l%d.mlp.e%d.%s" % (i, e, part)) for e in range(mlp["router"]["experts"])]
        out["layers"].append(w)
    return out


def dense_shapes(out, pre, ff, width):
    out[pre + "gate"] = out[pre + "up"] = (ff, width)
    out[pre + "down"] = (width, ff)


def check_shapes(tensors, want, free=lambda name: ()):
    """tensors has every tensor of want in its shape; free(name): axes that the configuration leaves to the tensor."""
    for name, shape in want.items():
        if name not in tensors:
            raise loader.ParameterError("missing tensor %s" % name)
        got = tuple(tensors[name].shape)
        if len(got) != len(shape) or any(g != s for k, (g, s) in enumerate(zip(got, shape)) if k not in free(name)):
            raise loader.ParameterError("%s has shape %s, the configuration says %s" % (name, list(got), list(shape)))


def upload(tensors, names):
    """{name: device bfloat16 array} of host arrays (bfloat16 bit patterns, or any float type, which is rounded)."""
    return {n: to_device(tensors[n] if tensors[n].dtype == np.uint16 else loader.to_bf16(tensors[n])) for n in names}


class HybridModel:
    """layers: list of dicts (HybridLayer fields).  weights: {"embed", "final_norm", "head": device bfloat16 arrays,
    "layers": list of dicts (HybridLayerWeights fields, experts as lists)}; they may be dropped once the model exists.
    embed_scale multiplies embedding rows; norm_add is added to the stored norm weights; post_norms: sublayers have a norm
    behind them; loop (start, stop, times): layers start .. stop-1 run `times` times in a row, each pass with rows and states
    of its own, the embedding output added ahead of every pass but the first.
    `slots` sequences of at most max_pos tokens each can be live at once."""

    def __init__(self, width, vocab, eps, layers, weights, dtype="bfloat16", max_pos=4096, slots=1, embed_scale=1.0, norm_add=0.0, post_norms=False,
                 loop=None):
        start, stop, times = loop or (0, 0, 1)
        # entries of the layer axis that step(layers=True) returns
        self.layer_runs = len(layers) + (stop - start) * (times - 1)
        self.width, self.vocab, self.max_pos, self.n_layers, self.dtype = int(width), int(vocab), int(max_pos), len(layers), dtype
        cfg = HybridConfig(layers=len(layers), width=self.width, vocab=self.vocab, max_pos=self.max_pos, slots=int(slots),
                           dtype=DTYPES[dtype], eps=float(eps),
                           embed_scale=float(embed_scale), norm_add=float(norm_add), post_norms=int(post_norms),
                           loop_start=int(start), loop_stop=int(stop), loop_times=int(times))
        ly = (HybridLayer * len(layers))()
        lw = (HybridLayerWeights * len(layers))()
        keep = []
        for i, d in enumerate(layers):
            ly[i].kv_from = -1
            for k, v in d.items():
                setattr(ly[i], k, v)
            for k, v in weights["layers"][i].items():
                if isinstance(v, (list, tuple)):
                    arr = (C.c_void_p * len(v))(*[a.ptr for a in v])
                    keep.append(arr)
                    setattr(lw[i], k, C.cast(arr, C.c_void_p))
                else:
                    setattr(lw[i], k, v.ptr)
        w = HybridWeights(*[weights[n].ptr for n in ("embed", "final_norm", "head")])
        h = C.c_void_p()
        self.handle = None
        check(lib().flexllm_hybrid_create(C.byref(h), C.byref(cfg), ly, C.byref(w), lw))
        self.handle = h
        self.pool = SlotPool(int(slots), self._reset)
        self._stream = None

    @classmethod
    def from_dir(cls, path, cfg, **kw):
        """cfg: the parsed config.json of the folder; from_tensors is the design's."""
        return cls.from_tensors(cfg, loader.read_safetensors(os.path.join(path, "model.safetensors")), **kw)

    # ---- sequences
    def _reset(self, slot):
        check(lib().flexllm_hybrid_reset(self.handle, int(slot), _s(self._stream)))

    def length(self, slot):
        n = C.c_int()
        check(lib().flexllm_hybrid_length(self.handle, int(slot), C.byref(n)))
        return n.value

    def stream(self):
        """The stream that everything of this model runs on."""
        if self._stream is None:
            self._stream = Stream()
        return self._stream

    # ---- steps
    def step(self, slot, tokens, want=(), layers=False):
        """Run `tokens` (host ids, or a device int32 array) of the slot's sequence; float32 logits [len(want)][vocab] of
        the wanted places (ascending), or None.  layers=True also returns the residual after every layer run."""
        st = self.stream()
        dev = tokens if isinstance(tokens, DeviceArray) else to_device(np.ascontiguousarray(tokens, np.int32).reshape(-1))
        want = np.ascontiguousarray(want, np.int32).reshape(-1)
        logits = DeviceArray((want.size, self.vocab), np.float32) if want.size else None
        res = DeviceArray((self.layer_runs, dev.size, self.width), np.float32) if layers else None
        check(lib().flexllm_hybrid_step(self.handle, int(slot), C.c_void_p(dev.ptr), dev.size,
                                        want.ctypes.data_as(C.c_void_p) if want.size else None, want.size,
                                        C.c_void_p(logits.ptr) if logits else None, C.c_void_p(res.ptr) if res else None, _s(st)))
        st.sync()
        out = logits.numpy() if logits else None
        return (out, res.numpy()) if layers else out

    def decode(self, slot, token_io, steps, tokens_out, rands=None, top_k=0, use_graph=True, stream=None):
        check(lib().flexllm_hybrid_decode(self.handle, int(slot), C.c_void_p(token_io.ptr), int(steps),
                                          C.c_void_p(rands.ptr) if rands is not None else None, int(top_k),
                                          C.c_void_p(tokens_out.ptr), int(use_graph), _s(stream or self.stream())))

    def generate(self, prompt, steps, top_k=0, rands=None, use_graph=True):
        """Prompt (host token ids) -> `steps` generated ids (host list), greedy (top_k = 0) or top-k sampling with the
        host-supplied uniform numbers `rands`, as llama.Llama.generate.  Takes a free slot for the time of the call."""
        prompt = np.ascontiguousarray(prompt, np.int32).reshape(-1)
        if top_k and rands is None:
            raise ValueError("top-k sampling needs `rands`, one uniform number in [0,1) per step")
        d_rands = to_device(np.ascontiguousarray(rands, np.float32).reshape(-1)) if top_k else None
        if top_k and d_rands.size < steps:
            raise ValueError("%d uniform numbers for %d steps" % (d_rands.size, steps))
        st = self.stream()
        d_prompt = to_device(prompt)
        out = DeviceArray((max(int(steps), 1),), np.int32)
        owner = object()
        slot = self.pool.acquire(owner)
        try:
            check(lib().flexllm_hybrid_generate(self.handle, slot, C.c_void_p(d_prompt.ptr), int(prompt.size), int(steps),
                                                C.c_void_p(d_rands.ptr) if top_k else None, int(top_k), C.c_void_p(out.ptr),
                                                int(use_graph), _s(st)))
            st.sync()
            self.check()
        finally:
            self.pool.release(owner)
        return out.numpy()[:int(steps)].tolist()

    def check(self):
        """Synchronise and raise if a token id outside the vocabulary was fed in."""
        check(lib().flexllm_hybrid_check(self.handle))

    def close(self):
        if self.handle:
            lib().flexllm_hybrid_destroy(self.handle)
            self.handle = None

    def __del__(self):
        try:
            self.close()
        except Exception:
            pass
