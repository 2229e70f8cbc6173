"""Plain, slow Turudra implementation: one function per mechanism, straight
from the design's equations, float64 by default, one sequence at a time.

It shares nothing with the package (it reads the raw config dict and a
name -> array mapping), so it can serve as the ground truth for the
kernels.  ``plant`` hooks let a test corrupt a mechanism on the CPU to
show that a comparison would notice.
"""

import math

import numpy as np


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def logsigmoid(z):
    return np.minimum(z, 0.0) - np.log1p(np.exp(-np.abs(z)))


def rotate_half(x, positions, base, dims):
    """x [T, ..., n]; the first ``dims`` of the last axis are rotated in
    pairs (i, i + dims/2) by position * base**(-2i/dims)."""
    half = dims // 2
    f = base ** (-2.0 * np.arange(half) / dims)
    a = np.asarray(positions, dtype=np.float64)[:, None] * f
    a = a.reshape((a.shape[0],) + (1,) * (x.ndim - 2) + (half,))
    c, s = np.cos(a), np.sin(a)
    u, v, rest = x[..., :half], x[..., half:dims], x[..., dims:]
    return np.concatenate([u * c - v * s, v * c + u * s, rest], axis=-1)


def latent_attention(w, p, m, h, eps, state):
    """h [T, width]; state holds the latents and rotated key parts of the
    tokens before h.  Returns (out [T, width], new state)."""
    H, d, r, vd = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    rank = m["kv_rank"]
    T = len(h)
    past = 0 if state is None else len(state[0])
    pos = past + np.arange(T)
    q = (h @ w[p + "q"].T).reshape(T, H, d + r)
    qr = rotate_half(q[..., d:], pos, m["rot"]["base"], m["rot"]["dims"])
    ckr = h @ w[p + "dkv"].T
    c = rms(ckr[:, :rank], eps) * w[p + "dkv.norm"]
    kr = rotate_half(ckr[:, rank:], pos, m["rot"]["base"], m["rot"]["dims"])
    if state is not None:
        c = np.concatenate([state[0], c])
        kr = np.concatenate([state[1], kr])
    k = (c @ w[p + "uk"].T).reshape(-1, H, d)
    v = (c @ w[p + "uv"].T).reshape(-1, H, vd)
    s = np.einsum("thd,jhd->htj", q[..., :d], k)
    s = (s + np.einsum("thd,jd->htj", qr, kr)) * m["scale"]
    see = np.arange(past + T)[None, :] <= pos[:, None]
    s = np.where(see[None], s, -np.inf)
    a = np.exp(s - s.max(axis=-1, keepdims=True))
    a /= a.sum(axis=-1, keepdims=True)
    o = np.einsum("htj,jhd->thd", a, v)
    o = o * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, H * vd) @ w[p + "o"].T, (c, kr)


def mlstm(w, p, m, h, eps, state):
    """Token-by-token matrix memory; state = (S, n, running maximum)."""
    H, d, vd, cap = m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    T = len(h)
    q = (h @ w[p + "q"].T).reshape(T, H, d) * d ** -0.5
    k = (h @ w[p + "k"].T).reshape(T, H, d)
    v = (h @ w[p + "v"].T).reshape(T, H, vd)
    li = cap * np.tanh((h @ w[p + "i"].T + w[p + "i.b"]) / cap)
    lf = logsigmoid(cap * np.tanh((h @ w[p + "f"].T + w[p + "f.b"]) / cap))
    if state is None:
        state = (np.zeros((H, d, vd)), np.zeros((H, d)), np.zeros(H))
    S, n, mx = state
    out = np.empty((T, H, vd), dtype=h.dtype)
    for t in range(T):
        new = np.maximum(lf[t] + mx, li[t])
        keep, add = np.exp(lf[t] + mx - new), np.exp(li[t] - new)
        S = keep[:, None, None] * S + add[:, None, None] * (
            k[t][:, :, None] * v[t][:, None, :])
        n = keep[:, None] * n + add[:, None] * k[t]
        mx = new
        num = np.einsum("hdv,hd->hv", S, q[t])
        den = np.maximum(np.abs((n * q[t]).sum(-1)), np.exp(-mx)) + 1e-6
        out[t] = num / den[:, None]
    y = rms(out, eps).reshape(T, H * vd) * w[p + "norm"]
    y = y * sigmoid(h @ w[p + "g"].T)
    return y @ w[p + "o"].T, (S, n, mx)


def expert(w, p, limit, h):
    g = np.minimum(h @ w[p + "gate"].T, limit)
    u = np.clip(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def route(z, top):
    """Indices [T, top] of the largest logits and their softmax."""
    idx = np.argsort(-z, axis=-1, kind="stable")[:, :top]
    zz = np.take_along_axis(z, idx, axis=-1)
    e = np.exp(zz - zz.max(axis=-1, keepdims=True))
    return idx, e / e.sum(axis=-1, keepdims=True)


def moe(w, p, c, h):
    idx, wt = route(h @ w[p + "router"].T, c["router"]["top"])
    y = np.zeros_like(h)
    for t in range(len(h)):
        for e, a in zip(idx[t], wt[t]):
            y[t] += a * expert(w, f"{p}e{e}.", c["expert"]["limit"],
                               h[t:t + 1])[0]
    if c.get("shared"):
        y = y + expert(w, p + "shared.", c["shared"]["limit"], h)
    return y


MIXERS = {"latent_attention": latent_attention, "mlstm": mlstm}


def layer_runs(cfg):
    """The layers in the order they run: (layer, starts a pass)."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    runs = [(i, False) for i in range(loop["start"])]
    for _ in range(loop["times"]):
        runs += [(i, i == loop["start"])
                 for i in range(loop["start"], loop["stop"])]
    return runs + [(i, False) for i in range(loop["stop"], n)]


class Oracle:
    def __init__(self, cfg, weights, dtype=np.float64):
        self.cfg = cfg
        self.w = {k: np.asarray(v).astype(dtype) for k, v in weights.items()}
        self.dtype = dtype

    def run(self, tokens, state=None, trace=None):
        """Logits [T, vocab] of ``tokens`` after ``state`` (a list with
        one entry per layer run, or None at the start); returns
        (logits, new state).  ``trace`` collects the residual."""
        cfg, w = self.cfg, self.w
        eps = cfg["norm"]["eps"]
        x = w["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
        x0 = x
        new = []
        for j, (i, starts) in enumerate(layer_runs(cfg)):
            if starts:
                x = np.concatenate([x, x0], axis=-1) @ w["loop.in"].T
            lc, p = cfg["layers"][i], f"l{i}."
            h = rms(x, eps) * w[p + "norm1"]
            y, st = MIXERS[lc["type"]](w, p + "mix.", lc["mixer"], h, eps,
                                       None if state is None else state[j])
            new.append(st)
            if lc.get("mlp"):
                y = y + moe(w, p + "mlp.", lc["mlp"], h)
            x = x + cfg["residual_mult"] * y
            if trace is not None:
                trace.append(x)
        z = (rms(x, eps) * w["final.norm"]) @ w["head"].T
        cap = cfg.get("logit_softcap")
        return (cap * np.tanh(z / cap) if cap else z), new
