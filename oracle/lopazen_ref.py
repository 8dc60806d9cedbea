"""Plain NumPy statement of the Lopazen decoder, one function per mechanism (test infrastructure only).

Nothing here is fast and nothing is shared with the device path: every mechanism is written out token by token from its
equation, in float64 by default.  `weights` maps tensor names to arrays, `cfg` is the parsed config.json dictionary."""
import math

import numpy as np


def rms_norm(x, weight, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * weight


def gelu(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def temperature(pos, coef, every):
    """Factor on the query at position pos: grows by coef * ln(n + 1) where n whole periods have passed."""
    return 1.0 + coef * math.log((pos + 1) // every + 1)


def sink_softmax(s):
    """exp(s_j) / (1 + sum exp(s)): one more key of score 0 that has no value."""
    top = max(float(s.max()), 0.0)
    e = np.exp(s - top)
    return e / (math.exp(-top) + e.sum())


def key_values(mx, w, pre, h, eps):
    """(normed keys, values) [T][kv heads][dim]: the values are the projected keys ahead of their norm."""
    k = (h @ w[pre + "k"].T + w[pre + "k.b"]).reshape(len(h), mx["kv_heads"], mx["dim"])
    return rms_norm(k, w[pre + "k.norm"], eps), k


def attention(mx, w, pre, h, pos0, keys, values, eps):
    """h [T][width] at positions pos0 ..; keys, values of positions 0 .. pos0+T-1."""
    H, G, d = mx["heads"], mx["kv_heads"], mx["dim"]
    q = (h @ w[pre + "q"].T + w[pre + "q.b"]).reshape(len(h), H, d)
    q = rms_norm(q, w[pre + "q.norm"], eps)
    out = np.zeros((len(h), H, mx["vdim"]), h.dtype)
    for t in range(len(h)):
        p = pos0 + t
        f = temperature(p, mx["q_temp"]["coef"], mx["q_temp"]["every"])
        for n in range(H):
            g = n // (H // G)
            a = sink_softmax(keys[:p + 1, g] @ (q[t, n] * f) * mx["scale"])
            out[t, n] = a @ values[:p + 1, g]
    return out.reshape(len(h), -1) @ w[pre + "o"].T


def feed_forward(w, pre, h):
    return (gelu(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def layer_runs(cfg):
    """[(layer, does this run open a repetition of the loop)] in the order in which the layers run."""
    n, lp = len(cfg["layers"]), cfg["loop"]
    out = [(i, False) for i in range(lp["start"])]
    for k in range(lp["times"]):
        out += [(i, k > 0 and i == lp["start"]) for i in range(lp["start"], lp["stop"])]
    return out + [(i, False) for i in range(lp["stop"], n)]


class Reference:
    """One sequence; `run` may be called with any number of tokens at a time."""

    def __init__(self, cfg, weights, dtype=np.float64):
        self.cfg = cfg
        self.w = {n: np.asarray(a).astype(dtype) for n, a in weights.items()}
        self.runs = layer_runs(cfg)
        self.reset()

    def reset(self):
        self.pos = 0
        self.held = [None] * len(self.runs)               # (keys, values) per layer run

    def run(self, tokens, trace=None):
        eps, w = self.cfg["norm"]["eps"], self.w
        first = w["embed"][np.asarray(tokens)] * self.cfg["embedding"]["scale"]
        x = first
        for r, (i, again) in enumerate(self.runs):
            ly, pre = self.cfg["layers"][i], "l%d." % i
            if again:
                x = x + first
            h = rms_norm(x, w[pre + "norm1"], eps)
            new = key_values(ly["mixer"], w, pre + "mix.", h, eps)
            self.held[r] = new if self.held[r] is None else tuple(np.concatenate(p) for p in zip(self.held[r], new))
            x = x + attention(ly["mixer"], w, pre + "mix.", h, self.pos, *self.held[r], eps)
            if ly.get("mlp"):
                x = x + feed_forward(w, pre + "mlp.", rms_norm(x, w[pre + "norm2"], eps))
            if trace is not None:
                trace.append(x.copy())
        self.pos += len(x)
        return rms_norm(x, w["final.norm"], eps) @ w["embed"].T
