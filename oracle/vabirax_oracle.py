"""Plain, slow restatement of the Vabirax design in numpy: one function per mechanism, whole sequences at a time, no cache, no
kernels and nothing shared with the product.  Test infrastructure only.

Everything is computed in `dtype` (float64 by default).  A model is a dict of tensors by checkpoint name and the parsed
config.json.
"""
import numpy as np


def dyn_tanh(x, alpha, w, b):
    """Dynamic Tanh: an elementwise squashing in the place of a norm, no statistics."""
    return np.tanh(alpha * x) * w + b


def rms(x, w, eps):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def rotate_half(x, pos, dims, base):
    """x [..., T, D]: dimension i < dims / 2 turns against dimension i + dims / 2 by the angle pos * base^(-2 i / dims)."""
    half = dims // 2
    inv = np.power(np.asarray(base, x.dtype), -2.0 * np.arange(half, dtype=x.dtype) / dims)
    ang = pos.astype(x.dtype)[:, None] * inv
    c, s = np.cos(ang), np.sin(ang)
    u, v = x[..., :half], x[..., half:dims]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., dims:]], axis=-1)


def window_mask(n, size):
    """mask[i, j]: may position i look at position j?  size None or 0: every earlier position."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    ok = j <= i
    if size:
        ok &= i - j < size
    return ok


def softmax_rows(s):
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def latent_attention(h, p, mix, eps):
    """h [T, width] -> [T, width].  p: the mixer's tensors by short name ('dq', 'dq.norm', ...)."""
    T = h.shape[0]
    H, d, r, dv = mix["heads"], mix["dim"], mix["rot_dim"], mix["vdim"]
    pos = np.arange(T)
    rot = mix["rot"]
    q = (rms(h @ p["dq"].T, p["dq.norm"], eps) @ p["uq"].T).reshape(T, H, d + r)
    kv = h @ p["dkv"].T
    c = rms(kv[:, :mix["kv_rank"]], p["dkv.norm"], eps)
    k_rot = rotate_half(kv[:, mix["kv_rank"]:], pos, rot["dims"], rot["base"])
    k = (c @ p["uk"].T).reshape(T, H, d)
    v = (c @ p["uv"].T).reshape(T, H, dv)
    ok = window_mask(T, (mix.get("mask") or {}).get("size"))
    out = np.empty((T, H, dv), h.dtype)
    for n in range(H):
        q_rot = rotate_half(q[:, n, d:], pos, rot["dims"], rot["base"])
        s = (q[:, n, :d] @ k[:, n].T + q_rot @ k_rot.T) * mix["scale"]
        out[:, n] = softmax_rows(np.where(ok, s, -np.inf)) @ v[:, n]
    return (out.reshape(T, H * dv) * sigmoid(h @ p["g"].T)) @ p["o"].T


def gated_ff(h, p):
    return (silu(h @ p["gate"].T) * (h @ p["up"].T)) @ p["down"].T


def loop_input(x, x0, w):
    return np.concatenate([x, x0], axis=-1) @ w.T


def layer_order(config):
    """[(layer index, first of a looped pass?)] in the order they run."""
    loop, n = config.get("loop"), len(config["layers"])
    if not loop:
        return [(i, False) for i in range(n)]
    body = [(i, i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return [(i, False) for i in range(loop["start"])] + body * loop["times"] + [(i, False) for i in range(loop["stop"], n)]


class Oracle:
    def __init__(self, config, tensors, dtype=np.float64):
        self.c = config
        self.dtype = dtype
        self.t = {k: np.asarray(v).astype(dtype) for k, v in tensors.items()}

    def norm(self, x, name):
        return dyn_tanh(x, self.t[name + ".alpha"], self.t[name], self.t[name + ".b"])

    def _part(self, prefix):
        return {k[len(prefix):]: v for k, v in self.t.items() if k.startswith(prefix)}

    def layer(self, x, i):
        L = self.c["layers"][i]
        if L["type"] != "latent_attention":
            raise ValueError(L["type"])
        n = "l%d." % i
        y = latent_attention(self.norm(x, n + "norm1"), self._part(n + "mix."), L["mixer"], self.c["norm"]["eps"])
        x = x + self.norm(y, n + "norm1b")
        if L["mlp"] is not None:
            y = gated_ff(self.norm(x, n + "norm2"), self._part(n + "mlp."))
            x = x + self.norm(y, n + "norm2b")
        return x

    def forward(self, tokens):
        """(logits [T, vocab], residual stream after every layer run [runs, T, width])"""
        x0 = self.t["embed"][np.asarray(tokens)] * self.dtype(self.c["embedding"]["scale"])
        x, runs = x0, []
        for i, first in layer_order(self.c):
            if first:
                x = loop_input(x, x0, self.t["loop.in"])
            x = self.layer(x, i)
            runs.append(x)
        return self.norm(x, "final.norm") @ self.t["head"].T, np.stack(runs)

    def greedy(self, prompt, n):
        ids = [int(t) for t in prompt]
        out = []
        for _ in range(n):
            lg = self.forward(ids)[0][-1]
            nxt = int(np.flatnonzero(lg == lg.max())[-1])
            ids.append(nxt)
            out.append(nxt)
        return out
