"""Plain, slow Dogalorn implementation: one function per mechanism, straight
from the design's equations, float64 by default, one sequence at a time.

It shares nothing with the package (it reads the raw config dict and a
name -> array mapping), so it can serve as the ground truth for the
kernels.  Mixers take and return their own state: keys and values so far,
recurrent states, last inputs of a convolution.
"""

import math

import numpy as np


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(z, np.zeros_like(z))


def gelu(z):
    return 0.5 * z * (1.0 + np.vectorize(math.erf)(z / math.sqrt(2.0)))


# ------------------------------------------------------------- embedding

def embed(w, spec, tokens, prev):
    """Token rows plus the rows of (previous, current) pairs; prev is the
    token before the first one (None at a sequence's start)."""
    x = w["embed"][tokens].copy()
    for t, cur in enumerate(tokens):
        before = tokens[t - 1] if t else prev
        if before is None:
            row = spec["buckets"]
        else:
            row = (int(before) * spec["mul_prev"] +
                   int(cur) * spec["mul_cur"]) % spec["buckets"]
        x[t] += w["bigram"][row]
    return x


# ------------------------------------------------------- streams of x

def gather(streams, weights):
    """What a sublayer reads: sum_s weights[s] x_s."""
    return sum(weights[s] * x for s, x in enumerate(streams))


def spread(streams, mix, out, y):
    """The streams after a sublayer with output y; mix is [from, to]."""
    n = len(streams)
    return [sum(mix[s, t] * streams[s] for s in range(n)) + out[t] * y
            for t in range(n)]


# ------------------------------------------------------------- attention

def bucket(n, rows, far):
    """Bucket of distance n: exact below rows/2, logarithmic up to far."""
    half = rows / 2
    if n < half:
        return n
    return int(min(rows - 1, half + math.floor(
        math.log(n / half) / math.log(far / half) * (rows - half))))


def visible(i, j, size):
    return j <= i and i // size == j // size


def sink_softmax(s):
    """One more term, of score 0 and without a value."""
    top = max(s.max(), 0.0)
    e = np.exp(s - top)
    return e / (e.sum() + np.exp(-top))


def attention(w, p, m, h, eps, past):
    H, G, d, size = m["heads"], m["kv_heads"], m["dim"], m["mask"]["size"]
    T = len(h)
    q, k = h @ w[p + "q"].T, h @ w[p + "k"].T
    v = k.reshape(T, G, d)
    q = (rms(q, eps) * w[p + "q.norm"]).reshape(T, H, d)
    k = (rms(k, eps) * w[p + "k.norm"]).reshape(T, G, d)
    n = 0 if past is None else len(past[0])
    if past is not None:
        k, v = np.concatenate([past[0], k]), np.concatenate([past[1], v])
    rel, temp = w[p + "rel"], w[p + "temp"]
    buckets = np.array([bucket(b, len(rel), m["bias_max"])
                        for b in range(min(n + T, size))])
    out = np.zeros((T, H, d), h.dtype)
    for t in range(T):
        i = n + t
        js = [j for j in range(i + 1) if visible(i, j, size)]
        bias = rel[buckets[i - np.array(js)]]
        for a in range(H):
            g = a // (H // G)
            s = k[js, g] @ q[t, a] * m["scale"] * temp[a] + bias[:, a]
            out[t, a] = sink_softmax(s) @ v[js, g]
    return out.reshape(T, H * d) @ w[p + "o"].T, (k, v)


# ------------------------------------------------------ gated recurrence

def candidate(u):
    return np.where(u >= 0, u + 0.5, sigmoid(u))


def mingru(w, p, m, h, eps, S):
    z = sigmoid(h @ w[p + "z"].T + w[p + "z.b"])
    c = candidate(h @ w[p + "x"].T + w[p + "x.b"])
    g = silu(h @ w[p + "g"].T)
    S = np.zeros(m["width"], h.dtype) if S is None else S
    y = np.empty_like(z)
    for t in range(len(h)):
        S = (1.0 - z[t]) * S + z[t] * c[t]
        y[t] = S * g[t]
    return y @ w[p + "o"].T, S


def halves(left, right, gl, gr, eps):
    return 0.5 * (rms(left, eps) * gl + rms(right, eps) * gr)


def parallel(w, p, m, h, eps, state):
    a, b = state or (None, None)
    left, a = attention(w, p + "left.", m["left"], h, eps, a)
    right, b = mingru(w, p + "right.", m["right"], h, eps, b)
    return halves(left, right, w[p + "left.out"], w[p + "right.out"],
                  eps), (a, b)


# ------------------------------------------------- state-space recurrence

def short_conv(x, w, b, before):
    """Causal convolution per channel, w [channels, taps]; ``before`` holds
    the taps - 1 inputs ahead of x (None: zeros)."""
    taps = w.shape[1]
    if before is None:
        before = np.zeros((taps - 1, x.shape[1]), x.dtype)
    full = np.concatenate([before, x])
    y = np.tile(b, (len(x), 1))
    for t in range(len(x)):
        for j in range(taps):
            y[t] = y[t] + w[:, j] * full[t + j]
    return y, full[len(full) - (taps - 1):]


def group_norm(y, g, groups, eps):
    T, n = y.shape
    return rms(y.reshape(T, groups, n // groups), eps).reshape(T, n) * g


def mamba2(w, p, m, h, eps, state):
    H, vd, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner, T = H * vd, len(h)
    S, before = state or (np.zeros((H, N, vd), h.dtype), None)
    z, xbc, dt = np.split(h @ w[p + "in"].T,
                          [inner, 2 * inner + 2 * G * N], axis=1)
    xbc, before = short_conv(xbc, w[p + "conv"], w[p + "conv.b"], before)
    x, B, C = np.split(silu(xbc), [inner, inner + G * N], axis=1)
    x = x.reshape(T, H, vd)
    B, C = B.reshape(T, G, N), C.reshape(T, G, N)
    dt = softplus(dt + w[p + "dt_bias"])
    rate = np.exp(w[p + "A_log"])
    S = S.copy()
    y = np.empty((T, H, vd), h.dtype)
    for t in range(T):
        for a in range(H):
            g = a // (H // G)
            S[a] = (np.exp(-rate[a] * dt[t, a]) * S[a] +
                    dt[t, a] * np.outer(B[t, g], x[t, a]))
            y[t, a] = S[a].T @ C[t, g] + w[p + "D"][a] * x[t, a]
    y = group_norm(y.reshape(T, inner) * silu(z), w[p + "norm"],
                   m["norm_groups"], eps)
    return y @ w[p + "o"].T, (S, before)


MIXERS = {"parallel": parallel, "mamba2": mamba2}


def dense(w, p, h):
    return gelu(h @ w[p + "up"].T + w[p + "up.b"]) @ w[p + "down"].T + \
        w[p + "down.b"]


# ----------------------------------------------------------------- model

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
        """Logits [T, vocab] of ``tokens`` after ``state`` (None at the
        start); returns (logits, new state).  ``trace`` collects the sum of
        the streams after every layer."""
        cfg, w = self.cfg, self.w
        eps = cfg["norm"]["eps"]
        tokens = np.asarray(tokens)
        prev, states = state or (None, [None] * len(cfg["layers"]))
        x = embed(w, cfg["embedding"]["bigram"], tokens, prev)
        xs = [x] * cfg["streams"]
        new = []
        for j, lc in enumerate(cfg["layers"]):
            p = f"l{owner(cfg, j)}."

            def sublayer(q, f):
                nonlocal xs
                c = f"{p}hc{q}."
                u = gather(xs, w[c + "in"])
                y = f(rms(u, eps) * w[f"{p}norm{q}"])
                xs = spread(xs, w[c + "mix"], w[c + "out"], y)

            def mixer(h):
                y, st = MIXERS[lc["type"]](w, p + "mix.", lc["mixer"], h, eps,
                                           states[j])
                new.append(st)
                return y

            sublayer(1, mixer)
            if lc.get("mlp"):
                sublayer(2, lambda h: dense(w, p + "mlp.", h))
            if trace is not None:
                trace.append(sum(xs))
        h = rms(sum(xs), eps) * w["final.norm"]
        return h @ w["head"].T * cfg["logit_scale"], (int(tokens[-1]), new)
