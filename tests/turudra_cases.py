"""Small random models for the Turudra tests."""

import numpy as np

from turudra_oracle import Oracle


def latent(heads=3, dim=20, rot=12, vdim=28, rank=40, dims=None, base=5e3,
           scale=None):
    return "latent_attention", dict(
        heads=heads, dim=dim, rot_dim=rot, vdim=vdim, kv_rank=rank,
        scale=scale or (dim + rot) ** -0.5,
        rot={"base": base, "dims": dims or rot})


def mlstm(heads=2, dim=36, vdim=52, cap=9.0):
    return "mlstm", dict(heads=heads, dim=dim, vdim=vdim, gate_cap=cap)


def moe(experts=5, top=2, ff=40, limit=1.3, shared=72, slimit=0.8):
    return {"kind": "moe", "router": {"experts": experts, "top": top},
            "expert": {"ff": ff, "limit": limit},
            "shared": {"ff": shared, "limit": slimit} if shared else None}


def config(layers, width=88, vocab=157, loop=None, eps=2e-5, emb=1.7,
           mult=0.45, cap=11.0):
    """layers: (mixer, mlp or None) pairs."""
    return {"architecture": "Turudra", "vocab": vocab, "width": width,
            "norm": {"eps": eps}, "embedding": {"scale": emb},
            "residual_mult": mult, "logit_softcap": cap,
            "loop": None if loop is None else dict(
                zip(("start", "stop", "times"), loop)),
            "layers": [{"type": m[0], "mixer": m[1], "mlp": f}
                       for m, f in layers]}


def default(**kw):
    """Every mechanism once, no two sizes alike."""
    return config([(latent(), moe()), (mlstm(), moe(4, 3, 72, 0.9, 24, 2.0)),
                   (latent(5, 12, 8, 16, 70, 6), None), (mlstm(3, 16, 80), moe(
                       6, 1, 16, 5.0, None))], loop=(1, 3, 2), **kw)


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
        elif name.endswith(".b"):
            a = 1.5 * a + (2.0 if ".f." in name else 0.0)
        elif name.endswith((".i", ".f")):
            a = 2.0 * a / np.sqrt(shape[-1])
        elif name.endswith("router"):
            a = 3.0 * a / np.sqrt(shape[-1])
        else:
            a = 1.4 * a / np.sqrt(shape[-1])
        w[name] = torch.from_numpy(a).to(torch.bfloat16).float().numpy()
    return w


def tokens(cfg, n, seed=0):
    return np.random.default_rng(100 + seed).integers(
        0, cfg["vocab"], size=n).astype(np.int32)


def rel(got, want):
    """Root mean square of the difference over that of the expectation."""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    assert got.shape == want.shape, (got.shape, want.shape)
    return float(np.sqrt(np.mean((got - want) ** 2) /
                         max(np.mean(want ** 2), 1e-30)))


def worst(got, want):
    """Largest per-row relative error, against the overall magnitude."""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    assert got.shape == want.shape, (got.shape, want.shape)
    s = max(np.sqrt(np.mean(want ** 2)), 1e-30)
    return float(np.sqrt(np.mean((got - want) ** 2, axis=-1)).max() / s)


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


def save(cfg, w, path):
    import json

    import torch
    from safetensors.torch import save_file

    path.mkdir(parents=True, exist_ok=True)
    (path / "config.json").write_text(json.dumps(cfg))
    save_file({k: torch.from_numpy(v).to(torch.bfloat16)
               for k, v in w.items()}, str(path / "model.safetensors"))
    return path
