"""Plain NumPy statement of the Nifunex decoder, one function per mechanism (test infrastructure only).

Nothing here is fast and nothing is shared with the device path: every mechanism is written out token by token from its
equation, in float64 by default.  `weights` maps tensor names to arrays, `cfg` is the parsed config.json dictionary."""
import math

import numpy as np


def rms(x, eps):
    return x / np.sqrt(np.mean(np.square(x), axis=-1, keepdims=True) + eps)


def norm_about_zero(x, w, eps):
    """RMS norm whose stored weight is the deviation from one."""
    return rms(x, eps) * (1.0 + w)


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def silu(z):
    return z * sigmoid(z)


def yarn_frequencies(rot):
    """(angular frequency per pair, factor on sine and cosine)."""
    dims, base = rot["dims"], rot["base"]
    i = np.arange(dims // 2, dtype=np.float64)
    f = base ** (-2.0 * i / dims)
    s = rot.get("scaling")
    if not s:
        return f, 1.0
    def turn_dim(t):
        return dims * math.log(s["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))
    lo = max(math.floor(turn_dim(s["fast"])), 0)
    hi = min(math.ceil(turn_dim(s["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / s["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(s["factor"]) + 1.0


def rotate_pairs(x, pos, rot):
    """x [..., dims] at position pos; neighbours (2i, 2i+1) form a pair."""
    f, m = yarn_frequencies(rot)
    c, s = m * np.cos(pos * f), m * np.sin(pos * f)
    u, v = x[..., 0::2], x[..., 1::2]
    out = np.empty_like(x)
    out[..., 0::2] = u * c - v * s
    out[..., 1::2] = v * c + u * s
    return out


def latent_rows(mx, w, pre, h, pos0, eps):
    """What a latent-attention layer stores per token: (normed latent, rotated shared key part)."""
    raw = h @ w[pre + "dkv"].T
    r = mx["kv_rank"]
    c = rms(raw[:, :r], eps) * w[pre + "dkv.norm"]
    k = np.stack([rotate_pairs(raw[t, r:], pos0 + t, mx["rot"]) for t in range(len(h))])
    return c, k


def latent_attention(mx, w, pre, h, pos0, c, k_rot):
    """h [T][width] at positions pos0..; c, k_rot: stored rows of positions 0 .. pos0+T-1."""
    H, d, rd, vd = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"]
    q = (h @ w[pre + "q"].T).reshape(len(h), H, d + rd)
    size = (mx.get("mask") or {}).get("size")
    out = np.zeros((len(h), H, vd), h.dtype)
    k_un = (c @ w[pre + "uk"].T).reshape(len(c), H, d)
    val = (c @ w[pre + "uv"].T).reshape(len(c), H, vd)
    for t in range(len(h)):
        p = pos0 + t
        lo = max(0, p - size + 1) if size else 0
        for n in range(H):
            qr = rotate_pairs(q[t, n, d:], p, mx["rot"])
            s = (k_un[lo:p + 1, n] @ q[t, n, :d] + k_rot[lo:p + 1] @ qr) * mx["scale"]
            e = np.exp(s - s.max())
            out[t, n] = (e / e.sum()) @ val[lo:p + 1, n]
    return out.reshape(len(h), -1) @ w[pre + "o"].T


def gla_decay_log(mx, w, pre, h):
    """log of the per-channel decay, [T][heads][dim]."""
    z = (h @ w[pre + "a1"].T) @ w[pre + "a2"].T + w[pre + "a2.b"]
    return (-np.logaddexp(0.0, -z) / mx["tau"]).reshape(len(h), mx["heads"], mx["dim"])


def gla_recurrence(q, k, v, log_a, state):
    """q, k, log_a [T][H][dim], v [T][H][vdim], state [H][dim][vdim] (updated in place).  Returns o [T][H][vdim]."""
    out = np.zeros(v.shape, v.dtype)
    for t in range(len(q)):
        for n in range(q.shape[1]):
            state[n] = np.exp(log_a[t, n])[:, None] * state[n] + np.outer(k[t, n], v[t, n])
            out[t, n] = state[n].T @ q[t, n]
    return out


def gla(mx, w, pre, h, state, eps):
    H, d, vd, T = mx["heads"], mx["dim"], mx["vdim"], len(h)
    q = (h @ w[pre + "q"].T).reshape(T, H, d) * d ** -0.5
    k = (h @ w[pre + "k"].T).reshape(T, H, d)
    v = (h @ w[pre + "v"].T).reshape(T, H, vd)
    o = gla_recurrence(q, k, v, gla_decay_log(mx, w, pre, h), state)
    o = rms(o, eps) * w[pre + "norm"]
    return (o.reshape(T, H * vd) * silu(h @ w[pre + "g"].T)) @ w[pre + "o"].T


def clamped_glu(g, u, limit):
    g = np.minimum(g, limit)
    u = np.clip(u, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


def feed_forward(w, pre, h, limit):
    return clamped_glu(h @ w[pre + "gate"].T, h @ w[pre + "up"].T, limit) @ w[pre + "down"].T


def route(scores_in, top):
    """Router outputs [E] -> (chosen experts, weights)."""
    e = np.exp(scores_in - scores_in.max())
    s = e / e.sum()
    pick = np.argsort(-s, kind="stable")[:top]
    return pick, s[pick] / (s[pick].sum() + 1e-20)


def mixture(mlp, w, pre, h):
    out = np.zeros_like(h)
    z = h @ w[pre + "router"].T
    for t in range(len(h)):
        pick, wt = route(z[t], mlp["router"]["top"])
        for e, a in zip(pick, wt):
            out[t] += a * feed_forward(w, "%se%d." % (pre, e), h[t:t + 1], mlp["expert"]["limit"])[0]
    if mlp.get("shared"):
        out = out + feed_forward(w, pre + "shared.", h, mlp["shared"]["limit"]) * sigmoid(h @ w[pre + "shared.sg"].T)
    return out


class Reference:
    """One sequence; `run` may be called with any number of tokens at a time."""

    def __init__(self, cfg, weights, dtype=np.float64):
        self.cfg, self.dtype = cfg, dtype
        self.w = {n: np.asarray(a).astype(dtype) for n, a in weights.items()}
        self.reset()

    def reset(self):
        self.pos = 0
        self.c, self.k, self.s = {}, {}, {}
        for i, ly in enumerate(self.cfg["layers"]):
            mx = ly["mixer"]
            if ly["type"] == "gla":
                self.s[i] = np.zeros((mx["heads"], mx["dim"], mx["vdim"]), self.dtype)
            elif mx.get("kv_from") is None:
                self.c[i] = np.zeros((0, mx["kv_rank"]), self.dtype)
                self.k[i] = np.zeros((0, mx["rot_dim"]), self.dtype)

    def run(self, tokens, trace=None):
        eps, w = self.cfg["norm"]["eps"], self.w
        x = w["embed"][np.asarray(tokens)]
        for i, ly in enumerate(self.cfg["layers"]):
            pre, mx = "l%d." % i, ly["mixer"]
            h = norm_about_zero(x, w[pre + "norm1"], eps)
            if ly["type"] == "gla":
                y = gla(mx, w, pre + "mix.", h, self.s[i], eps)
            else:
                j = mx.get("kv_from")
                if j is None:
                    j = i
                    c, k = latent_rows(mx, w, pre + "mix.", h, self.pos, eps)
                    self.c[i], self.k[i] = np.concatenate([self.c[i], c]), np.concatenate([self.k[i], k])
                y = latent_attention(mx, w, pre + "mix.", h, self.pos, self.c[j], self.k[j])
            x = x + norm_about_zero(y, w[pre + "norm1b"], eps)
            mlp = ly.get("mlp")
            if mlp:
                h = norm_about_zero(x, w[pre + "norm2"], eps)
                if mlp["kind"] == "dense":
                    y = feed_forward(w, pre + "mlp.", h, mlp["limit"])
                else:
                    y = mixture(mlp, w, pre + "mlp.", h)
                x = x + norm_about_zero(y, w[pre + "norm2b"], eps)
            if trace is not None:
                trace.append(x.copy())
        self.pos += len(x)
        return norm_about_zero(x, w["final.norm"], eps) @ w["head"].T
