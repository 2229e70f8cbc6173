"""Small random models for the Dogalorn tests."""

import numpy as np

from dogalorn_oracle import Oracle
from turudra_cases import rel, save, tokens, worst  # noqa: F401  (re-exported)


def attention(heads=4, kv_heads=2, dim=20, chunk=45, far=30, scale=None):
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim,
                scale=scale or dim ** -0.5, bias_max=far,
                mask={"size": chunk})


def pair(heads=4, kv_heads=2, dim=20, chunk=45, far=30, width=92, scale=None):
    return "parallel", {"left": attention(heads, kv_heads, dim, chunk, far,
                                          scale), "right": {"width": width}}


def ssd(heads=6, vdim=20, state=28, groups=3, conv=4, norm_groups=2):
    return "mamba2", dict(heads=heads, vdim=vdim, state=state, groups=groups,
                          conv=conv, norm_groups=norm_groups)


def dense(ff=112):
    return {"kind": "dense", "ff": ff}


def config(layers, width=88, vocab=157, streams=3, eps=2e-5, logit_scale=0.6,
           buckets=211, muls=(31, 7)):
    """layers: (mixer, feed-forward or None[, layer whose tensors it uses])."""
    return {"architecture": "Dogalorn", "vocab": vocab, "width": width,
            "norm": {"eps": eps}, "streams": streams,
            "logit_scale": logit_scale,
            "embedding": {"bigram": {"buckets": buckets, "mul_prev": muls[0],
                                     "mul_cur": muls[1]}},
            "layers": [{"type": m[0], "mixer": m[1], "mlp": f,
                        **({"weights_of": of[0]} if of else {})}
                       for m, f, *of in layers]}


def default(**kw):
    """Every mechanism, no two sizes alike; layers 4 and 6 use the tensors
    of layers 0 and 1, layer 5 those of layer 4."""
    a = (pair(), dense())
    b = (ssd(), dense(72))
    return config([a, b, (pair(3, 3, 36, 70, 90, 40), None),
                   (ssd(4, 36, 20, 1, 3, 3), dense(130)),
                   (*a, 0), (*a, 4), (*b, 1), (ssd(2, 68, 76, 2, 2, 1), None)],
                  **kw)


def weights(cfg, seed=0, buckets=10):
    """float32 arrays, rounded to bf16 values so both dtypes of the engine
    and the oracle see the same numbers; `buckets` rows of distance biases."""
    import torch

    from llm_np_cp_amd.core.layered import LayeredConfig

    rng = np.random.default_rng(seed)
    w = {}
    for name, shape in LayeredConfig.from_dict(cfg).weight_shapes().items():
        if name.endswith(".rel"):
            shape = (buckets, shape[1])
        a = rng.standard_normal(shape)
        if ".hc" in name:
            a = 0.3 * a + (np.eye(*shape) if name.endswith("mix") else
                           1 / shape[0] if name.endswith("in") else 1.0)
        elif "norm" in name or name.endswith(("left.out", "right.out")):
            a = 1.0 + 0.2 * a
        elif name in ("embed", "bigram"):
            a = 0.7 * a
        elif name.endswith("z.b"):
            a = a - 3.0            # decays near 1: the state reaches back
        elif name.endswith("A_log"):
            a = a - 1.5
        elif name.endswith("dt_bias"):
            a = a - 2.0
        elif name.endswith(("temp", ".D")):
            a = 1.0 + 0.3 * a
        elif name.endswith((".b", "conv")):
            a = 0.6 * a
        elif not name.endswith(".rel"):
            a = 1.4 * a / np.sqrt(shape[-1])
        w[name] = torch.from_numpy(np.asarray(a)).to(
            torch.bfloat16).float().numpy()
    return w


def greedy(cfg, w, prompt, n):
    """n greedy tokens by the oracle, and the smallest top-2 margin."""
    o, ids, margin = Oracle(cfg, w), [], np.inf
    z, st = o.run(prompt)
    for _ in range(n):
        two = np.sort(z[-1])[-2:]
        margin = min(margin, two[1] - two[0])
        ids.append(int(np.argmax(z[-1])))
        z, st = o.run([ids[-1]], st)
    return ids, margin


def only(cfg, w, half):
    """The pairs' other half silenced, and no token pairs."""
    for k in w:
        if k.endswith({"left": "right.out", "right": "left.out"}[half]):
            w[k] = w[k] * 0
    w["bigram"] = w["bigram"] * 0
    return w


def needle(at, total, chunk, heads=4, kv_heads=4, dim=24, far=40):
    """A model and prompt in which the last token attends to one position
    almost alone: only token 1, placed there, has the key that only token
    2, placed last, asks for.  Nothing else carries it forward."""
    cfg = config([(pair(heads, kv_heads, dim, chunk, far), None)], width=64,
                 streams=2)
    w = only(cfg, weights(cfg, 9), "left")
    w["embed"][:, :8] = 0
    w["embed"][2, :4] = w["embed"][1, 4:8] = 6.0
    d = np.random.default_rng(2).choice([-1.0, 1.0], dim).astype(np.float32)
    for name, lo in (("q", 0), ("k", 4)):
        m = w["l0.mix.left." + name]
        m[:, :8] = 0
        m[:, lo:lo + 4] = np.tile(d, len(m) // dim)[:, None]
        w[f"l0.mix.left.{name}.norm"][:] = 1
    w["l0.mix.left.temp"][:] = 2.0
    t = 3 + tokens(cfg, total) % (cfg["vocab"] - 3)
    t[at], t[-1] = 1, 2
    return cfg, w, t.astype(np.int32)


def memory(kind, total):
    """A one-layer model and prompt whose recurrence takes up the first
    token only and then keeps it; another first token shows at the end."""
    cfg = config([(pair() if kind == "mingru" else ssd(), None)], streams=2)
    w = only(cfg, weights(cfg, 3), "right")
    w["embed"][:, 0] = 0
    w["embed"][5:7, 0] = 9.0
    if kind == "mingru":
        gate, b, m = w["l0.mix.right.z"], "l0.mix.right.z.b", 3.0
    else:
        gate, b, m = w["l0.mix.in"][-6:], "l0.mix.dt_bias", 2.0
        w["l0.mix.A_log"][:] = -3.0
        w["l0.mix.D"] *= 0
    gate *= 0
    gate[:, 0] = m
    w[b][:] = -9.0
    t = 7 + tokens(cfg, total) % (cfg["vocab"] - 7)
    t[0] = 5
    return cfg, w, t.astype(np.int32)
