"""Plain, slow Fidizen implementation: one function per mechanism, straight
from the design's equations, float64 by default, one sequence at a time.

It shares nothing with the package (it reads the raw config dict and a
name -> array mapping), so it can serve as the ground truth for the
kernels.  Sublayers take and return their own state: the latents and
rotated keys so far, and the last inputs of the convolution ahead of them.
"""

import numpy as np


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def short_conv(h, w, before):
    """h + a causal convolution per channel, w [channels, taps]; ``before``
    holds the taps - 1 inputs ahead of h (None: zeros)."""
    taps = w.shape[1]
    if before is None:
        before = np.zeros((taps - 1, h.shape[1]), h.dtype)
    full = np.concatenate([before, h])
    y = h.copy()
    for t in range(len(h)):
        for j in range(taps):
            y[t] += w[:, j] * full[t + j]
    return y, full[len(full) - (taps - 1):]


def rotate(x, pos, base, dims):
    """Pairs (2i, 2i+1) of the first ``dims`` of x [T, ..., n] turn by
    pos * base^(-2i/dims)."""
    x = x.copy()
    for i in range(dims // 2):
        a = pos * base ** (-2.0 * i / dims)
        a = a.reshape((-1,) + (1,) * (x.ndim - 2))
        u, v = x[..., 2 * i].copy(), x[..., 2 * i + 1].copy()
        x[..., 2 * i] = u * np.cos(a) - v * np.sin(a)
        x[..., 2 * i + 1] = v * np.cos(a) + u * np.sin(a)
    return x


def visible(pos, keys, window):
    """[T, J]: a token sees itself and the window - 1 tokens before it."""
    back = pos[:, None] - np.arange(keys)[None]
    return (back >= 0) & (back < window)


def sink_softmax(s, sink):
    """s [T, J], -inf where hidden; one more term in the denominator."""
    top = np.maximum(s.max(axis=-1, keepdims=True), sink)
    e = np.exp(s - top)
    return e / (e.sum(axis=-1, keepdims=True) + np.exp(sink - top))


def latent_attention(w, p, m, h, eps, past):
    H, d, r, vd, rank = (m[k] for k in ("heads", "dim", "rot_dim", "vdim",
                                        "kv_rank"))
    T, n = len(h), 0 if past is None else len(past[0])
    pos = n + np.arange(T)
    base, dims = m["rot"]["base"], m["rot"]["dims"]
    q = (rms(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]) @ w[p + "uq"].T
    q = q.reshape(T, H, d + r)
    qr = rotate(q[..., d:], pos, base, dims)
    ckv = h @ w[p + "dkv"].T
    c = rms(ckv[:, :rank], eps) * w[p + "dkv.norm"]
    kr = rotate(ckv[:, rank:], pos, base, dims)
    if past is not None:
        c, kr = np.concatenate([past[0], c]), np.concatenate([past[1], kr])
    see = visible(pos, n + T, m["mask"]["size"])
    out = np.empty((T, H, vd), h.dtype)
    for i in range(H):
        k = c @ w[p + "uk"][i * d:(i + 1) * d].T
        v = c @ w[p + "uv"][i * vd:(i + 1) * vd].T
        s = (q[:, i, :d] @ k.T + qr[:, i] @ kr.T) * m["scale"]
        out[:, i] = sink_softmax(np.where(see, s, -np.inf),
                                 w[p + "sink"][i]) @ v
    out = out.reshape(T, H * vd) * sigmoid(h @ w[p + "g"].T)
    return out @ w[p + "o"].T, (c, kr)


def polynorm(z, coef, eps):
    a, b, c, e = coef
    return a * rms(z, eps) + b * rms(z ** 2, eps) + c * rms(z ** 3, eps) + e


def dense(w, p, m, h, eps):
    return polynorm(h @ w[p + "up"].T, w[p + "act"], eps) @ w[p + "down"].T


def expert(w, p, h):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def choose(z, top):
    """The experts with the largest scores, and those scores."""
    s = sigmoid(z)
    idx = np.argsort(-s, kind="stable")[:top]
    return idx, s[idx]


def moe(w, p, m, h, eps):
    z = h @ w[p + "router"].T
    y = np.zeros_like(h)
    for t in range(len(h)):
        for e, s in zip(*choose(z[t], m["router"]["top"])):
            y[t] += expert(w, f"{p}e{e}.", s * h[t])
        if m.get("shared"):
            y[t] += expert(w, p + "shared.", h[t])
    return y


FEED_FORWARDS = {"dense": dense, "moe": moe}


def owner(cfg, i):
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


class Oracle:
    def __init__(self, cfg, weights, dtype=np.float64):
        self.cfg = cfg
        self.w = {k: np.asarray(v).astype(dtype) for k, v in weights.items()}

    def run(self, tokens, state=None, trace=None):
        """Logits [T, vocab] of ``tokens`` after ``state`` (a list with
        one entry per layer, or None at the start); returns
        (logits, new state).  ``trace`` collects the residual."""
        cfg, w = self.cfg, self.w
        eps = cfg["norm"]["eps"]
        x = w["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
        new = []
        for j, lc in enumerate(cfg["layers"]):
            p = f"l{owner(cfg, j)}."
            past, c1, c2 = (None,) * 3 if state is None else state[j]
            h, c1 = short_conv(x, w[p + "canon1"], c1)
            y, past = latent_attention(w, p + "mix.", lc["mixer"], h, eps,
                                       past)
            x = x + rms(y, eps) * w[p + "norm1"]
            if lc.get("mlp"):
                h, c2 = short_conv(x, w[p + "canon2"], c2)
                y = FEED_FORWARDS[lc["mlp"]["kind"]](w, p + "mlp.", lc["mlp"],
                                                     h, eps)
                x = x + rms(y, eps) * w[p + "norm2"]
            new.append((past, c1, c2))
            if trace is not None:
                trace.append(x)
        return (rms(x, eps) * w["final.norm"]) @ w["head"].T, new
