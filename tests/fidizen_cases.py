"""Small random models for the Fidizen tests."""

import numpy as np

from fidizen_oracle import Oracle
from turudra_cases import rel, save, tokens, worst  # noqa: F401  (re-exported)


def latent(heads=3, dim=20, rot=12, vdim=28, rank=40, q_rank=36, window=45,
           base=5e3, scale=None):
    return dict(heads=heads, dim=dim, rot_dim=rot, vdim=vdim, kv_rank=rank,
                q_rank=q_rank, scale=scale or (dim + rot) ** -0.5,
                mask={"size": window}, rot={"base": base, "dims": rot})


def dense(ff=112):
    return {"kind": "dense", "ff": ff}


def moe(experts=5, top=2, ff=40, shared=72):
    return {"kind": "moe", "router": {"experts": experts, "top": top},
            "expert": {"ff": ff}, "shared": {"ff": shared} if shared else None}


def config(layers, width=88, vocab=157, taps=3, eps=2e-5, emb=1.7):
    """layers: (mixer, feed-forward or None[, layer whose tensors it uses])."""
    return {"architecture": "Fidizen", "vocab": vocab, "width": width,
            "norm": {"eps": eps}, "embedding": {"scale": emb},
            "canon": {"taps": taps},
            "layers": [{"type": "latent_attention", "mixer": m, "mlp": f,
                        **({"weights_of": of[0]} if of else {})}
                       for m, f, *of in layers]}


def default(**kw):
    """Every mechanism, no two sizes alike; layers 3 and 5 use the tensors
    of layers 0 and 1, layer 4 those of layer 3."""
    a = (latent(), dense())
    b = (latent(5, 12, 8, 16, 70, 52, 64, 900.0), moe())
    c = (latent(2, 36, 20, 44, 24, 100, 21, scale=0.3), None)
    return config([a, b, c, (*a, 0), (*a, 3), (*b, 1),
                   (latent(window=1000), moe(6, 3, 24, None))], **kw)


def weights(cfg, seed=0):
    """float32 arrays, rounded to bf16 values so both dtypes of the engine
    and the oracle see the same numbers."""
    import torch

    from llm_np_cp_amd.core.layered import LayeredConfig

    rng = np.random.default_rng(seed)
    w = {}
    for name, shape in LayeredConfig.from_dict(cfg).weight_shapes().items():
        a = rng.standard_normal(shape)
        if "norm" in name:
            a = 1.0 + 0.2 * a
        elif name == "embed":
            a = 0.7 * a
        elif "canon" in name:
            a = 0.5 * a
        elif name.endswith("sink"):
            a = 1.0 + 1.5 * a
        elif name.endswith("act"):
            a = np.array([0.6, -0.5, 0.3, 0.2]) + 0.1 * a
        elif name.endswith("router"):
            a = 2.0 * a / np.sqrt(shape[-1])
        else:
            a = 1.4 * a / np.sqrt(shape[-1])
        w[name] = torch.from_numpy(a).to(torch.bfloat16).float().numpy()
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


def needle(at, total, window, heads=4, rank=40, q_rank=36):
    """A model and prompt in which the last token attends to one position
    almost alone: only token 1, placed there, has the key that only token
    2, placed last, asks for.  Without convolutions, so that nothing else
    carries it forward."""
    cfg = config([(latent(heads, 24, 12, 40, rank, q_rank, window), None)],
                 width=64, taps=2)
    w = weights(cfg, 9)
    w["l0.canon1"] *= 0
    w["l0.mix.sink"][:] = 1.0
    w["embed"][:, :8] = 0
    w["embed"][2, :4] = w["embed"][1, 4:8] = 6.0
    d = np.random.default_rng(2).choice([-1.0, 1.0], 24).astype(np.float32)
    for name, lo in (("dq", 0), ("dkv", 4)):    # component 0 marks the token
        m = w["l0.mix." + name]
        m[:, :8] = 0
        m[0] = 0
        m[0, lo:lo + 4] = 2.0
        w[f"l0.mix.{name}.norm"][:] = 1
    uq = w["l0.mix.uq"].reshape(heads, 36, q_rank)
    uq[:, :24, 0], uq[:, 24:, 0] = d / 2, 0
    w["l0.mix.uk"].reshape(heads, 24, rank)[:, :, 0] = d / 2
    t = 3 + tokens(cfg, total) % (cfg["vocab"] - 3)
    t[at], t[-1] = 1, 2
    return cfg, w, t.astype(np.int32)
