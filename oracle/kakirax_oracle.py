"""Plain, slow restatement of the Kakirax design in numpy: one function per mechanism, whole sequences at a time, no cache, no
kernels and nothing shared with the product.  Test infrastructure only.

Everything is computed in `dtype` (float64 by default).  A model is a dict of tensors by checkpoint name and the parsed
config.json.
"""
import math

import numpy as np


def layer_norm(x, w, b, eps):
    """Centred and scaled by the standard deviation (mean of the squared deviations), then an affine map."""
    d = x - x.mean(axis=-1, keepdims=True)
    return d / np.sqrt((d * d).mean(axis=-1, keepdims=True) + eps) * w + b


def rms(x, w, eps):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps) * w


def sigmoid(z):
    return np.where(z >= 0, 1.0, np.exp(np.minimum(z, 0))) / (1.0 + np.exp(-np.abs(z)))


def log_sigmoid(z):
    return np.minimum(z, 0) - np.log1p(np.exp(-np.abs(z)))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def frequencies(dims, base, scaling, dtype=np.float64):
    """Angle per position of each rotated pair.  scaling (or None): waves longer than original / low are slowed by `factor`, waves
    shorter than original / high stay, and those between are blended by where their number of turns in `original` lies."""
    f = np.power(np.asarray(base, dtype), -2.0 * np.arange(dims // 2, dtype=dtype) / dims)
    if scaling is None:
        return f
    out = []
    for w in f:
        length = 2.0 * math.pi / w
        if length < scaling["original"] / scaling["high"]:
            out.append(w)
        elif length > scaling["original"] / scaling["low"]:
            out.append(w / scaling["factor"])
        else:
            s = (scaling["original"] / length - scaling["low"]) / (scaling["high"] - scaling["low"])
            out.append((1.0 - s) * w / scaling["factor"] + s * w)
    return np.asarray(out, dtype)


def rotate_half(x, pos, dims, freq):
    """x [..., T, D]: dimension i < dims / 2 turns against dimension i + dims / 2 by pos * freq[i]; the rest passes."""
    half = dims // 2
    ang = pos.astype(x.dtype)[:, None] * freq.astype(x.dtype)
    c, s = np.cos(ang), np.sin(ang)
    u, v = x[..., :half], x[..., half:dims]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., dims:]], axis=-1)


def softmax_rows(s):
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def attention(h, p, mix, eps):
    """Grouped-query attention with normed queries and keys and a sigmoid gate on the concatenated heads.
    h [T, width] -> [T, width].  p: the mixer's tensors by short name ('q', 'q.norm', ...)."""
    T = h.shape[0]
    H, G, d, dv, rot = mix["heads"], mix["kv_heads"], mix["dim"], mix["vdim"], mix["rot"]
    pos, freq = np.arange(T), frequencies(rot["dims"], rot["base"], rot.get("scaling"), h.dtype)
    q = rms((h @ p["q"].T).reshape(T, H, d), p["q.norm"], eps)
    k = rms((h @ p["k"].T).reshape(T, G, d), p["k.norm"], eps)
    v = (h @ p["v"].T).reshape(T, G, dv)
    later = np.arange(T)[None, :] > np.arange(T)[:, None]
    out = np.empty((T, H, dv), h.dtype)
    for n in range(H):
        g = n // (H // G)
        s = rotate_half(q[:, n], pos, rot["dims"], freq) @ rotate_half(k[:, g], pos, rot["dims"], freq).T * mix["scale"]
        out[:, n] = softmax_rows(np.where(later, -np.inf, s)) @ v[:, g]
    return (out.reshape(T, H * dv) * sigmoid(h @ p["g"].T)) @ p["o"].T


def decays(h, p, mix):
    """[T, heads, dim] in (0, 1]: sigmoid of a low-rank map, to the power 1 / tau."""
    z = (h @ p["a1"].T) @ p["a2"].T + p["a2.b"]
    return np.exp(log_sigmoid(z) / mix["tau"]).reshape(h.shape[0], mix["heads"], mix["dim"])


def gated_state(q, k, v, a):
    """The recurrence, token by token: S <- diag(a_t) S + k_t v_t^T, o_t = S^T q_t.  [T, heads, dim] x3 and v [T, heads, vdim]."""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]), q.dtype)
    out = np.empty(v.shape, q.dtype)
    for t in range(T):
        S = a[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (q[t][:, :, None] * S).sum(axis=1)
    return out


def gated_linear_attention(h, p, mix, eps):
    T = h.shape[0]
    H, d, dv = mix["heads"], mix["dim"], mix["vdim"]
    q = (h @ p["q"].T).reshape(T, H, d) * d ** -0.5
    k = (h @ p["k"].T).reshape(T, H, d)
    v = (h @ p["v"].T).reshape(T, H, dv)
    o = rms(gated_state(q, k, v, decays(h, p, mix)), p["norm"], eps)
    return (o.reshape(T, H * dv) * silu(h @ p["g"].T)) @ p["o"].T


def gated_ff(h, p):
    return (gelu_tanh(h @ p["gate"].T) * (h @ p["up"].T)) @ p["down"].T


def softcap(x, cap):
    return cap * np.tanh(x / cap)


MIXERS = {"attention": attention, "gla": gated_linear_attention}


class Oracle:
    def __init__(self, config, tensors, dtype=np.float64):
        self.c = config
        self.dtype = dtype
        self.eps = config["norm"]["eps"]
        self.t = {k: np.asarray(v).astype(dtype) for k, v in tensors.items()}

    def norm(self, x, name):
        return layer_norm(x, self.t[name], self.t[name + ".b"], self.eps)

    def part(self, prefix):
        return {k[len(prefix):]: v for k, v in self.t.items() if k.startswith(prefix)}

    def layer(self, x, i):
        L = self.c["layers"][i]
        owner = L.get("weights_of")
        n = "l%d." % (i if owner is None else owner)
        x = x + MIXERS[L["type"]](self.norm(x, n + "norm1"), self.part(n + "mix."), L["mixer"], self.eps)
        if L["mlp"] is not None:
            x = x + gated_ff(self.norm(x, n + "norm2"), self.part(n + "mlp."))
        return x

    def forward(self, tokens):
        """(logits [T, vocab], residual stream after every layer [layers, T, width])"""
        x = self.t["embed"][np.asarray(tokens)] * self.dtype(self.c["embedding"]["scale"])
        runs = []
        for i in range(len(self.c["layers"])):
            x = self.layer(x, i)
            runs.append(x)
        return softcap(self.norm(x, "final.norm") @ self.t["embed"].T, self.c["logit_softcap"]), np.stack(runs)

    def greedy(self, prompt, n):
        ids = [int(t) for t in prompt]
        out = []
        for _ in range(n):
            lg = self.forward(ids)[0][-1]
            nxt = int(np.flatnonzero(lg == lg.max())[-1])
            ids.append(nxt)
            out.append(nxt)
        return out
