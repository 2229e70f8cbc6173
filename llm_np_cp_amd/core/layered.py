"""Configuration of layer-list designs.

Where ``ModelConfig`` describes a stack of identical blocks, a layer-list
``config.json`` names every layer: its mixer, the mixer's sizes, its
feed-forward, and optionally a range of layers that runs several times.
Each mechanism is a small spec class that reads its own keys and knows its
tensors; a further design lists its specs under its name in ``DESIGNS``.

Turudra: parallel blocks (one norm feeds mixer and experts), latent
attention and matrix-memory LSTM mixers, clamped routed experts with a
shared one, a looped range that mixes the embedding output back in, and a
soft-capped head.

Garupel: sandwich blocks (a norm before and after each sublayer), grouped
attention without rotation, gated linear recurrence and decaying linear
attention mixers, dense feed-forwards, a looped range to which the
embedding output is added ahead of every pass but the first.

Fidizen: post-norm blocks (a norm on each sublayer's output only) whose
sublayers read the residual through a short causal convolution, latent
attention with a query latent, a sliding window and a sink, polynomial
dense feed-forwards or sigmoid-routed experts, layers that use another
layer's tensors.

Dogalorn: several residual streams that every sublayer reads and rewrites
through small learned mixes, an embedding of token pairs, pairs of mixers
side by side (chunked attention with distance biases whose values are its
keys, a gated recurrence), state-space mixers, biased gelu feed-forwards,
norms with a single gain, shared tensors.
"""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional, Tuple

import numpy as np

Shapes = Dict[str, Tuple[int, ...]]


def _get(d: dict, key: str, where: str):
    if not isinstance(d, dict) or key not in d:
        raise ValueError(f"config.json: {where} lacks {key!r}")
    return d[key]


def _positive(where: str, **kw):
    for k, v in kw.items():
        if isinstance(v, bool) or not isinstance(v, int) or v < 1:
            raise ValueError(f"config.json: {where}.{k} must be a positive "
                             f"integer, got {v!r}")


@dataclass
class LatentAttentionSpec:
    libs = ("latent",)
    recurrent = False
    inputs = ("q", "dkv", "g")   # matrices that read the mixer's input
    interleaved = False          # rotation pairs (i, i + dims/2)
    gate = "head"                # the output gate is one number per head
    q_rank = window = None       # no query latent, every earlier key
    sink = False
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot_base: float
    rot_dims: int
    kind = "latent_attention"

    @classmethod
    def from_dict(cls, m: dict, where: str):
        rot = _get(m, "rot", where)
        s = cls(heads=_get(m, "heads", where), dim=_get(m, "dim", where),
                rot_dim=_get(m, "rot_dim", where),
                vdim=_get(m, "vdim", where),
                kv_rank=_get(m, "kv_rank", where),
                scale=float(_get(m, "scale", where)),
                rot_base=float(_get(rot, "base", where + ".rot")),
                rot_dims=_get(rot, "dims", where + ".rot"))
        _positive(where, heads=s.heads, dim=s.dim, rot_dim=s.rot_dim,
                  vdim=s.vdim, kv_rank=s.kv_rank, rot_dims=s.rot_dims)
        if s.rot_dims % 2 or s.rot_dims > s.rot_dim:
            raise ValueError(f"config.json: {where}.rot.dims {s.rot_dims} "
                             f"must be even and at most {s.rot_dim}")
        return s

    def to_dict(self) -> dict:
        return {"heads": self.heads, "dim": self.dim,
                "rot_dim": self.rot_dim, "vdim": self.vdim,
                "kv_rank": self.kv_rank, "scale": self.scale,
                "rot": {"base": self.rot_base, "dims": self.rot_dims}}

    def shapes(self, p: str, width: int) -> Shapes:
        H = self.heads
        return {p + "q": (H * (self.dim + self.rot_dim), width),
                p + "dkv": (self.kv_rank + self.rot_dim, width),
                p + "dkv.norm": (self.kv_rank,),
                p + "uk": (H * self.dim, self.kv_rank),
                p + "uv": (H * self.vdim, self.kv_rank),
                p + "g": (H, width),
                p + "o": (width, H * self.vdim)}


@dataclass
class WindowedLatentSpec(LatentAttentionSpec):
    """Latent attention whose queries go through a latent of their own
    (q_rank), over the last `window` tokens, with a sink per head in the
    softmax, interleaved rotation and an output gate per element."""
    inputs = ("dq", "dkv", "g")
    interleaved = True
    gate = "element"
    sink = True
    q_rank: int = 0
    window: int = 0

    @classmethod
    def from_dict(cls, m: dict, where: str):
        s = super().from_dict(m, where)
        s.q_rank = _get(m, "q_rank", where)
        s.window = _get(_get(m, "mask", where), "size", where + ".mask")
        _positive(where, q_rank=s.q_rank)
        _positive(where + ".mask", size=s.window)
        return s

    def to_dict(self) -> dict:
        return {**super().to_dict(), "q_rank": self.q_rank,
                "mask": {"size": self.window}}

    def shapes(self, p: str, width: int) -> Shapes:
        out = super().shapes(p, width)
        H, Q = self.heads, self.q_rank
        out.pop(p + "q")
        out.update({p + "dq": (Q, width), p + "dq.norm": (Q,),
                    p + "uq": (H * (self.dim + self.rot_dim), Q),
                    p + "sink": (H,), p + "g": (H * self.vdim, width)})
        return out


@dataclass
class MLSTMSpec:
    libs = ("mlstm",)
    recurrent = True
    heads: int
    dim: int
    vdim: int
    gate_cap: float
    kind = "mlstm"

    @classmethod
    def from_dict(cls, m: dict, where: str):
        s = cls(heads=_get(m, "heads", where), dim=_get(m, "dim", where),
                vdim=_get(m, "vdim", where),
                gate_cap=float(_get(m, "gate_cap", where)))
        _positive(where, heads=s.heads, dim=s.dim, vdim=s.vdim)
        return s

    def to_dict(self) -> dict:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim,
                "gate_cap": self.gate_cap}

    def shapes(self, p: str, width: int) -> Shapes:
        H, qk, v = self.heads, self.heads * self.dim, self.heads * self.vdim
        return {p + "q": (qk, width), p + "k": (qk, width),
                p + "v": (v, width), p + "g": (v, width),
                p + "o": (width, v), p + "norm": (v,),
                p + "i": (H, width), p + "i.b": (H,),
                p + "f": (H, width), p + "f.b": (H,)}


@dataclass
class ExpertSpec:
    """W_down (act(W_gate h, W_up h)), act = silu(gate) up."""
    ff: int
    limit = 0.0

    @classmethod
    def from_dict(cls, m: dict, where: str):
        s = cls(ff=_get(m, "ff", where))
        _positive(where, ff=s.ff)
        return s

    def to_dict(self) -> dict:
        return {"ff": self.ff}

    def shapes(self, p: str, width: int) -> Shapes:
        return {p + "gate": (self.ff, width), p + "up": (self.ff, width),
                p + "down": (width, self.ff)}


@dataclass
class ClampedExpertSpec(ExpertSpec):
    """The GLU clamps both halves at `limit`."""
    limit: float = 0.0

    @classmethod
    def from_dict(cls, m: dict, where: str):
        s = super().from_dict(m, where)
        s.limit = float(_get(m, "limit", where))
        return s

    def to_dict(self) -> dict:
        return {"ff": self.ff, "limit": self.limit}


@dataclass
class MoESpec:
    """Routed experts and an optional shared one.  The chosen experts'
    weights are the softmax over their logits, applied to the outputs."""
    experts: int
    top: int
    expert: ExpertSpec
    shared: Optional[ExpertSpec] = None
    kind = "moe"
    libs = ("moe",)
    expert_class = ClampedExpertSpec
    glu = "clamped"
    score = "softmax"
    weigh = "output"

    @classmethod
    def from_dict(cls, m: dict, where: str):
        r = _get(m, "router", where)
        sh = m.get("shared")
        s = cls(experts=_get(r, "experts", where + ".router"),
                top=_get(r, "top", where + ".router"),
                expert=cls.expert_class.from_dict(
                    _get(m, "expert", where), where + ".expert"),
                shared=(cls.expert_class.from_dict(sh, where + ".shared")
                        if sh else None))
        _positive(where + ".router", experts=s.experts, top=s.top)
        if s.top > s.experts or s.experts > 1024:
            raise ValueError(f"config.json: {where}.router: top {s.top} of "
                             f"{s.experts} experts (at most 1024) is not "
                             f"possible")
        return s

    def to_dict(self) -> dict:
        return {"kind": self.kind,
                "router": {"experts": self.experts, "top": self.top},
                "expert": self.expert.to_dict(),
                "shared": self.shared.to_dict() if self.shared else None}

    def shapes(self, p: str, width: int) -> Shapes:
        out = {p + "router": (self.experts, width)}
        for e in range(self.experts):
            out.update(self.expert.shapes(f"{p}e{e}.", width))
        if self.shared:
            out.update(self.shared.shapes(p + "shared.", width))
        return out


@dataclass
class SigmoidMoESpec(MoESpec):
    """Every expert has a score sigmoid(logit); the scores of the chosen
    ones, as they are, weigh the experts' inputs."""
    expert_class = ExpertSpec
    glu = "silu"
    score = "sigmoid"
    weigh = "input"


@dataclass
class AttentionSpec:
    """Grouped-query attention without rotation: biased projections, RMS
    norm over the whole query and key projections, a query temperature
    1 + coef ln(floor((p + 1) / every) + 1), an output gate per element."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    temp_coef: float
    temp_every: int
    kind = "attention"
    libs = ("gqa",)
    recurrent = False
    inputs = ("q", "k", "v", "g")
    chunk = bias_max = None
    sink = False

    @classmethod
    def from_dict(cls, m: dict, where: str):
        qt = _get(m, "q_temp", where)
        s = cls(heads=_get(m, "heads", where),
                kv_heads=_get(m, "kv_heads", where),
                dim=_get(m, "dim", where), vdim=_get(m, "vdim", where),
                scale=float(_get(m, "scale", where)),
                temp_coef=float(_get(qt, "coef", where + ".q_temp")),
                temp_every=_get(qt, "every", where + ".q_temp"))
        _positive(where, heads=s.heads, kv_heads=s.kv_heads, dim=s.dim,
                  vdim=s.vdim)
        if s.heads % s.kv_heads:
            raise ValueError(f"config.json: {where}: {s.heads} heads do not "
                             f"divide over {s.kv_heads} kv_heads")
        if not s.temp_every > 0:
            raise ValueError(f"config.json: {where}.q_temp.every must be "
                             f"positive, got {s.temp_every!r}")
        return s

    def to_dict(self) -> dict:
        return {"heads": self.heads, "kv_heads": self.kv_heads,
                "dim": self.dim, "vdim": self.vdim, "scale": self.scale,
                "q_temp": {"coef": self.temp_coef, "every": self.temp_every}}

    def shapes(self, p: str, width: int) -> Shapes:
        q, k = self.heads * self.dim, self.kv_heads * self.dim
        v, o = self.kv_heads * self.vdim, self.heads * self.vdim
        return {p + "q": (q, width), p + "q.b": (q,), p + "q.norm": (q,),
                p + "k": (k, width), p + "k.b": (k,), p + "k.norm": (k,),
                p + "v": (v, width), p + "v.b": (v,), p + "g": (o, width),
                p + "o": (width, o)}


@dataclass
class ChunkedAttentionSpec:
    """Grouped-query attention without rotation, bias or gate.  A token sees
    the earlier ones of its chunk of `chunk` positions; the values are the
    keys ahead of their norm.  Scores are multiplied by a number per head
    and get a bias by distance, from a table whose rows are buckets: exact
    below half of them, logarithmic up to bias_max.  The softmax has one
    more term, of score 0."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    bias_max: float
    chunk: int
    kind = "attention"
    libs = ("gqa",)
    recurrent = False
    inputs = ("q", "k")
    sink = True
    buckets = 32                 # of random weights; a checkpoint has its own

    @classmethod
    def from_dict(cls, m: dict, where: str):
        s = cls(heads=_get(m, "heads", where),
                kv_heads=_get(m, "kv_heads", where),
                dim=_get(m, "dim", where), vdim=_get(m, "vdim", where),
                scale=float(_get(m, "scale", where)),
                bias_max=_get(m, "bias_max", where),
                chunk=_get(_get(m, "mask", where), "size", where + ".mask"))
        _positive(where, heads=s.heads, kv_heads=s.kv_heads, dim=s.dim,
                  vdim=s.vdim)
        _positive(where + ".mask", size=s.chunk)
        if s.heads % s.kv_heads:
            raise ValueError(f"config.json: {where}: {s.heads} heads do not "
                             f"divide over {s.kv_heads} kv_heads")
        if s.dim != s.vdim:
            raise ValueError(f"config.json: {where}: the values are the keys, "
                             f"but dim {s.dim} is not vdim {s.vdim}")
        if not s.bias_max > 0:
            raise ValueError(f"config.json: {where}.bias_max must be "
                             f"positive, got {s.bias_max!r}")
        return s

    def to_dict(self) -> dict:
        return {"heads": self.heads, "kv_heads": self.kv_heads,
                "dim": self.dim, "vdim": self.vdim, "scale": self.scale,
                "bias_max": self.bias_max, "mask": {"size": self.chunk}}

    def shapes(self, p: str, width: int) -> Shapes:
        q, k = self.heads * self.dim, self.kv_heads * self.dim
        return {p + "q": (q, width), p + "q.norm": (q,),
                p + "k": (k, width), p + "k.norm": (k,),
                p + "rel": (self.buckets, self.heads),
                p + "temp": (self.heads,), p + "o": (width, q)}

    def open_rows(self, p: str):
        return [p + "rel"]


@dataclass
class MinGRUSpec:
    """Gated recurrence whose gate and candidate read the current token
    only, element by element."""
    width: int
    kind = "mingru"
    libs = ("mingru",)
    recurrent = True
    inputs = ("z", "x", "g")

    @classmethod
    def from_dict(cls, m: dict, where: str):
        s = cls(width=_get(m, "width", where))
        _positive(where, width=s.width)
        return s

    def to_dict(self) -> dict:
        return {"width": self.width}

    def shapes(self, p: str, width: int) -> Shapes:
        C = self.width
        return {p + "z": (C, width), p + "z.b": (C,), p + "x": (C, width),
                p + "x.b": (C,), p + "g": (C, width), p + "o": (width, C)}


@dataclass
class PairSpec:
    """Two mixers that read the same input; the result is half the sum of
    their normed outputs."""
    left: object
    right: object
    kind = "parallel"
    left_class = ChunkedAttentionSpec
    right_class = MinGRUSpec

    @property
    def libs(self):
        return (*self.left.libs, *self.right.libs)

    @property
    def recurrent(self):
        return self.left.recurrent or self.right.recurrent

    @classmethod
    def from_dict(cls, m: dict, where: str):
        return cls(*(c.from_dict(_get(m, k, where), f"{where}.{k}")
                     for k, c in (("left", cls.left_class),
                                  ("right", cls.right_class))))

    def to_dict(self) -> dict:
        return {"left": self.left.to_dict(), "right": self.right.to_dict()}

    def shapes(self, p: str, width: int) -> Shapes:
        return {**self.left.shapes(p + "left.", width),
                **self.right.shapes(p + "right.", width),
                p + "left.out": (width,), p + "right.out": (width,)}

    def open_rows(self, p: str):
        return [n for k in ("left", "right")
                for n in open_rows(getattr(self, k), f"{p}{k}.")]


def open_rows(spec, p: str):
    """Tensors of a mixer whose number of rows the checkpoint decides."""
    return spec.open_rows(p) if hasattr(spec, "open_rows") else []


@dataclass
class SSDSpec:
    """State-space recurrence (Mamba-2): x, B and C behind a causal
    convolution of `conv` taps, a step size per head and token, the state a
    [state, vdim] matrix per head; the gated output is normed in
    norm_groups equal parts."""
    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int
    kind = "mamba2"
    libs = ("ssd",)
    recurrent = True
    inputs = ("in",)

    @classmethod
    def from_dict(cls, m: dict, where: str):
        names = ("heads", "vdim", "state", "groups", "conv", "norm_groups")
        s = cls(**{k: _get(m, k, where) for k in names})
        _positive(where, **{k: getattr(s, k) for k in names})
        if s.heads % s.groups:
            raise ValueError(f"config.json: {where}: {s.heads} heads do not "
                             f"divide over {s.groups} groups")
        if s.inner % s.norm_groups:
            raise ValueError(f"config.json: {where}: {s.inner} values do not "
                             f"divide into {s.norm_groups} norm_groups")
        return s

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def channels(self) -> int:
        """What passes the convolution: x, B and C."""
        return self.inner + 2 * self.groups * self.state

    def to_dict(self) -> dict:
        return {"heads": self.heads, "vdim": self.vdim, "state": self.state,
                "groups": self.groups, "conv": self.conv,
                "norm_groups": self.norm_groups}

    def shapes(self, p: str, width: int) -> Shapes:
        H, C = self.heads, self.channels
        return {p + "in": (self.inner + C + H, width),
                p + "conv": (C, self.conv), p + "conv.b": (C,),
                p + "dt_bias": (H,), p + "A_log": (H,), p + "D": (H,),
                p + "norm": (self.inner,), p + "o": (width, self.inner)}


@dataclass
class RGLRUSpec:
    """Two branches of `width`: a gelu one, and a causal convolution of
    `conv` taps feeding the real-gated linear recurrence, whose gates are
    block-diagonal over `blocks` parts."""
    width: int
    blocks: int
    conv: int
    kind = "rglru"
    libs = ("rglru",)
    recurrent = True
    C = 8.0                      # log a = -C r softplus(lam)

    @classmethod
    def from_dict(cls, m: dict, where: str):
        s = cls(width=_get(m, "width", where),
                blocks=_get(m, "blocks", where), conv=_get(m, "conv", where))
        _positive(where, width=s.width, blocks=s.blocks, conv=s.conv)
        if s.width % s.blocks:
            raise ValueError(f"config.json: {where}: width {s.width} does "
                             f"not divide into {s.blocks} blocks")
        return s

    def to_dict(self) -> dict:
        return {"width": self.width, "blocks": self.blocks,
                "conv": self.conv}

    def shapes(self, p: str, width: int) -> Shapes:
        C, nb, bw = self.width, self.blocks, self.width // self.blocks
        return {p + "y": (C, width), p + "y.b": (C,), p + "x": (C, width),
                p + "x.b": (C,), p + "conv": (C, self.conv),
                p + "conv.b": (C,), p + "ra": (nb, bw, bw),
                p + "ra.b": (nb, bw), p + "ri": (nb, bw, bw),
                p + "ri.b": (nb, bw), p + "lam": (C,), p + "o": (width, C)}


@dataclass
class LightningSpec:
    """Linear attention with a fixed decay per head."""
    heads: int
    dim: int
    vdim: int
    decay: List[float]
    kind = "lightning"
    libs = ("lightning",)
    recurrent = True

    @classmethod
    def from_dict(cls, m: dict, where: str):
        s = cls(heads=_get(m, "heads", where), dim=_get(m, "dim", where),
                vdim=_get(m, "vdim", where),
                decay=[float(x) for x in _get(m, "decay", where)])
        _positive(where, heads=s.heads, dim=s.dim, vdim=s.vdim)
        if len(s.decay) != s.heads or not all(0 <= x <= 1 for x in s.decay):
            raise ValueError(f"config.json: {where}.decay must hold "
                             f"{s.heads} numbers from 0 to 1")
        return s

    def to_dict(self) -> dict:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim,
                "decay": list(self.decay)}

    def shapes(self, p: str, width: int) -> Shapes:
        qk, v = self.heads * self.dim, self.heads * self.vdim
        return {p + "q": (qk, width), p + "k": (qk, width),
                p + "v": (v, width), p + "g": (v, width),
                p + "o": (width, v), p + "norm": (v,)}


@dataclass
class DenseSpec:
    """W_down act(W_up h), act = the square of relu."""
    ff: int
    kind = "dense"
    libs = ()
    act = "relu2"

    @classmethod
    def from_dict(cls, m: dict, where: str):
        s = cls(ff=_get(m, "ff", where))
        _positive(where, ff=s.ff)
        return s

    def to_dict(self) -> dict:
        return {"kind": self.kind, "ff": self.ff}

    def shapes(self, p: str, width: int) -> Shapes:
        return {p + "up": (self.ff, width), p + "down": (width, self.ff)}


@dataclass
class PolyDenseSpec(DenseSpec):
    """act(z) = a N(z) + b N(z^2) + c N(z^3) + e with learned a, b, c, e;
    N divides a token's vector by its root mean square."""
    act = "polynorm"

    def shapes(self, p: str, width: int) -> Shapes:
        return {**super().shapes(p, width), p + "act": (4,)}


@dataclass
class GeluDenseSpec(DenseSpec):
    """act = the exact gelu; both matrices have biases."""
    act = "gelu"

    def shapes(self, p: str, width: int) -> Shapes:
        return {**super().shapes(p, width), p + "up.b": (self.ff,),
                p + "down.b": (width,)}


@dataclass
class BigramSpec:
    """Embedding of token pairs: row (previous * mul_prev + current *
    mul_cur) mod buckets; one more row for a sequence's first token."""
    buckets: int
    mul_prev: int
    mul_cur: int

    @classmethod
    def from_dict(cls, m: dict, where: str):
        names = ("buckets", "mul_prev", "mul_cur")
        s = cls(**{k: _get(m, k, where) for k in names})
        _positive(where, **{k: getattr(s, k) for k in names})
        return s

    def to_dict(self) -> dict:
        return {"buckets": self.buckets, "mul_prev": self.mul_prev,
                "mul_cur": self.mul_cur}


@dataclass(frozen=True)
class Design:
    """What a design fixes about its layers.  ``parallel``: one norm feeds
    mixer and feed-forward; ``sandwich``: each has a norm before and after
    it; ``post``: each has a norm after it and a short convolution over
    time ahead of it; ``hyper``: each reads a mix of several residual
    streams through a norm with one gain and rewrites them all.
    ``project``: W_in [x; x0] ahead of every pass of the
    loop; ``add``: x + x0 ahead of every pass but the first.  ``share``: a
    layer may use another one's tensors."""
    model_type: str
    block: str
    loop: Optional[str]
    mixers: Tuple[type, ...]
    mlps: Tuple[type, ...]
    share: bool = False

    def mixer(self, kind):
        return next((c for c in self.mixers if c.kind == kind), None)

    def mlp(self, kind):
        return next((c for c in self.mlps if c.kind == kind), None)


# config "architecture" -> design
DESIGNS = {
    "Turudra": Design("turudra", "parallel", "project",
                      (LatentAttentionSpec, MLSTMSpec), (MoESpec,)),
    "Garupel": Design("garupel", "sandwich", "add",
                      (AttentionSpec, RGLRUSpec, LightningSpec),
                      (DenseSpec,)),
    "Fidizen": Design("fidizen", "post", None, (WindowedLatentSpec,),
                      (PolyDenseSpec, SigmoidMoESpec), share=True),
    "Dogalorn": Design("dogalorn", "hyper", None, (PairSpec, SSDSpec),
                       (GeluDenseSpec,), share=True),
}


@dataclass
class LayerSpec:
    mixer: object
    mlp: Optional[object]
    weights_of: Optional[int] = None   # the layer whose tensors it uses


@dataclass
class LoopSpec:
    start: int
    stop: int
    times: int


@dataclass
class LayeredConfig:
    model_type: str
    vocab_size: int
    hidden_size: int
    layers: List[LayerSpec]
    loop: Optional[LoopSpec] = None
    norm_eps: float = 1e-5
    embed_scale: float = 1.0
    residual_mult: float = 1.0
    logit_softcap: Optional[float] = None
    conv_taps: int = 1            # of the sublayers' input convolutions
    streams: int = 0              # copies of the residual, 0: it is plain
    bigram: Optional[BigramSpec] = None
    logit_scale: float = 1.0
    max_position_embeddings: int = 131072
    bos_token_id: Optional[int] = None
    eos_token_id: Optional[int] = None
    # (layer whose tensors run, the embedding output comes in ahead of it)
    runs: List[Tuple[int, bool]] = field(default_factory=list)

    def __post_init__(self):
        n, lp = len(self.layers), self.loop
        if lp is None:
            self.runs = [(self._owner(i), False) for i in range(n)]
            return
        if not (0 <= lp.start < lp.stop <= n and lp.times >= 1):
            raise ValueError(f"config.json: loop {lp} does not fit "
                             f"{n} layers")
        self.runs = [(i, False) for i in range(lp.start)]
        first = 0 if self.design.loop == "project" else 1
        for k in range(lp.times):
            self.runs += [(i, i == lp.start and k >= first)
                          for i in range(lp.start, lp.stop)]
        self.runs += [(i, False) for i in range(lp.stop, n)]

    def _owner(self, i: int) -> int:
        """The layer whose tensors layer i uses."""
        seen = [i]
        while self.layers[i].weights_of is not None:
            j = self.layers[i].weights_of
            if (isinstance(j, bool) or not isinstance(j, int) or
                    not 0 <= j < len(self.layers) or j in seen):
                raise ValueError(f"config.json: layers[{i}].weights_of {j!r} "
                                 f"is not possible")
            a, b = self.layers[seen[0]], self.layers[j]
            if (a.mixer, a.mlp) != (b.mixer, b.mlp):
                raise ValueError(f"config.json: layers[{seen[0]}] differs "
                                 f"from layers[{j}], whose tensors it uses")
            seen.append(j)
            i = j
        return i

    @property
    def architecture(self) -> str:
        return next(k for k, v in DESIGNS.items()
                    if v.model_type == self.model_type)

    @property
    def design(self) -> Design:
        return DESIGNS[self.architecture]

    def kernel_libraries(self) -> Tuple[str, ...]:
        """The kernel libraries that this list of layers launches."""
        libs = {"linear"}
        for l in self.layers:
            libs.update(l.mixer.libs)
            if l.mlp:
                libs.update(l.mlp.libs)
            elif self.design.block == "parallel":
                libs.add("moe")           # its fused output step
        return tuple(sorted(libs))

    # names the rest of the framework reads
    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @property
    def rms_norm_eps(self) -> float:
        return self.norm_eps

    @property
    def is_moe(self) -> bool:
        return any(l.mlp and l.mlp.kind == "moe" for l in self.layers)

    @property
    def recurrent(self) -> bool:
        return (self.conv_taps > 1 or self.bigram is not None or
                any(l.mixer.recurrent for l in self.layers))

    @classmethod
    def matches(cls, d: dict) -> bool:
        return "architecture" in d

    @classmethod
    def from_dict(cls, d: dict) -> "LayeredConfig":
        arch = _get(d, "architecture", "top level")
        if arch not in DESIGNS:
            raise ValueError(f"unsupported architecture {arch!r}; layer-list "
                             f"designs: {sorted(DESIGNS)}")
        design, layers = DESIGNS[arch], []
        for i, l in enumerate(_get(d, "layers", "top level")):
            w = f"layers[{i}]"
            kind = _get(l, "type", w)
            if design.mixer(kind) is None:
                raise ValueError(f"config.json: {w}: unknown mixer {kind!r}")
            mlp = l.get("mlp")
            if mlp is not None and design.mlp(mlp.get("kind")) is None:
                raise ValueError(f"config.json: {w}: unknown feed-forward "
                                 f"{mlp.get('kind')!r}")
            share = l.get("weights_of")
            if share is not None and not design.share:
                raise ValueError(f"config.json: {w}: {arch} does not share "
                                 f"tensors between layers")
            layers.append(LayerSpec(
                design.mixer(kind).from_dict(_get(l, "mixer", w),
                                             w + ".mixer"),
                design.mlp(mlp["kind"]).from_dict(mlp, w + ".mlp") if mlp
                else None, share))
        lp = d.get("loop")
        if lp and not design.loop:
            raise ValueError(f"config.json: {arch} has no loop")
        taps = 1
        if design.block == "post":
            taps = _get(_get(d, "canon", "top level"), "taps", "canon")
            _positive("canon", taps=taps)
        streams, bigram, logit_scale = 0, None, 1.0
        if design.block == "hyper":
            streams = _get(d, "streams", "top level")
            _positive("top level", streams=streams)
            bigram = BigramSpec.from_dict(
                _get(_get(d, "embedding", "top level"), "bigram",
                     "embedding"), "embedding.bigram")
            logit_scale = float(_get(d, "logit_scale", "top level"))
        width, vocab = _get(d, "width", "top level"), _get(d, "vocab",
                                                           "top level")
        _positive("top level", width=width, vocab=vocab)
        cap = d.get("logit_softcap")
        return cls(
            model_type=design.model_type, vocab_size=vocab, hidden_size=width,
            layers=layers,
            loop=LoopSpec(_get(lp, "start", "loop"), _get(lp, "stop", "loop"),
                          _get(lp, "times", "loop")) if lp else None,
            norm_eps=float(_get(_get(d, "norm", "top level"), "eps", "norm")),
            embed_scale=float(d.get("embedding", {}).get("scale", 1.0)),
            residual_mult=float(d.get("residual_mult", 1.0)),
            logit_softcap=float(cap) if cap else None,
            conv_taps=taps, streams=streams, bigram=bigram,
            logit_scale=logit_scale,
            max_position_embeddings=d.get("max_position_embeddings", 131072),
            bos_token_id=d.get("bos_token_id"),
            eos_token_id=d.get("eos_token_id"))

    def to_dict(self) -> dict:
        d = {"architecture": self.architecture, "vocab": self.vocab_size,
             "width": self.hidden_size, "norm": {"eps": self.norm_eps},
             "layers": [{"type": l.mixer.kind, "mixer": l.mixer.to_dict(),
                         "mlp": l.mlp.to_dict() if l.mlp else None}
                        for l in self.layers]}
        for entry, l in zip(d["layers"], self.layers):
            if l.weights_of is not None:
                entry["weights_of"] = l.weights_of
        if self.design.loop:
            d["loop"] = None
        if self.design.block == "post":
            d.update({"embedding": {"scale": self.embed_scale},
                      "canon": {"taps": self.conv_taps}})
        if self.design.block == "hyper":
            d.update({"embedding": {"bigram": self.bigram.to_dict()},
                      "streams": self.streams,
                      "logit_scale": self.logit_scale})
        if self.design.block == "parallel":
            d.update({"embedding": {"scale": self.embed_scale},
                      "residual_mult": self.residual_mult,
                      "logit_softcap": self.logit_softcap})
        if self.loop:
            d["loop"] = {"start": self.loop.start, "stop": self.loop.stop,
                         "times": self.loop.times}
        for k in ("bos_token_id", "eos_token_id"):
            if getattr(self, k) is not None:
                d[k] = getattr(self, k)
        return d

    to_hf_dict = to_dict

    def weight_shapes(self) -> Shapes:
        W = self.hidden_size
        out: Shapes = {"embed": (self.vocab_size, W), "final.norm": (W,),
                       "head": (self.vocab_size, W)}
        if self.loop and self.design.loop == "project":
            out["loop.in"] = (W, 2 * W)
        sandwich = self.design.block == "sandwich"
        post = self.design.block == "post"
        S, hyper = self.streams, self.design.block == "hyper"
        if hyper:
            out["final.norm"] = ()
        if self.bigram:
            out["bigram"] = (self.bigram.buckets + 1, W)
        for i, l in enumerate(self.layers):
            if l.weights_of is not None:
                continue
            out[f"l{i}.norm1"] = () if hyper else (W,)
            if hyper:
                if l.mlp:
                    out[f"l{i}.norm2"] = ()
                for q in (1, 2) if l.mlp else (1,):
                    out.update({f"l{i}.hc{q}.in": (S,), f"l{i}.hc{q}.out": (S,),
                                f"l{i}.hc{q}.mix": (S, S)})
            if post:
                out[f"l{i}.canon1"] = (W, self.conv_taps)
                if l.mlp:
                    out[f"l{i}.norm2"] = (W,)
                    out[f"l{i}.canon2"] = (W, self.conv_taps)
            if sandwich:
                out[f"l{i}.norm1b"] = (W,)
            out.update(l.mixer.shapes(f"l{i}.mix.", W))
            if l.mlp:
                if sandwich:
                    out[f"l{i}.norm2"] = out[f"l{i}.norm2b"] = (W,)
                out.update(l.mlp.shapes(f"l{i}.mlp.", W))
        return out

    def open_rows(self):
        """Names of tensors whose number of rows the checkpoint decides."""
        return {n for i, l in enumerate(self.layers) if l.weights_of is None
                for n in open_rows(l.mixer, f"l{i}.mix.")}

    def weight_base(self, name: str, shape):
        """What random weights scatter around: 1 for norms, streams that
        stay as they are and are read evenly."""
        if ".hc" in name:
            return (np.eye(*shape) if name.endswith("mix") else
                    np.full(shape, 1.0 / shape[0] if name.endswith("in")
                            else 1.0))
        return 1.0 if "norm" in name or name.endswith(
            ("left.out", "right.out")) else 0.0


# ----------------------------------------------------------------------
# presets (random-init runs)
# ----------------------------------------------------------------------

def _layer(mixer: str, experts: int, top: int, ff: int, shared: int,
           limit: float = 7.0, **m) -> dict:
    mlp = {"kind": "moe", "router": {"experts": experts, "top": top},
           "expert": {"ff": ff, "limit": limit},
           "shared": {"ff": shared, "limit": limit} if shared else None}
    return {"type": mixer, "mixer": m, "mlp": mlp if experts else None}


def _latent(heads, dim, rot, vdim, rank, base=10000.0) -> dict:
    return dict(heads=heads, dim=dim, rot_dim=rot, vdim=vdim, kv_rank=rank,
                scale=(dim + rot) ** -0.5, rot={"base": base, "dims": rot})


def _design(vocab, width, layers, loop=None, **kw) -> dict:
    d = {"architecture": "Turudra", "vocab": vocab, "width": width,
         "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
         "residual_mult": 0.5, "logit_softcap": 30.0, "layers": layers,
         "loop": loop}
    d.update(kw)
    return d


def _moe_stack(n, mix, width, heads, moe) -> list:
    """n layers: latent attention, or alternating with mLSTM (mix "both")."""
    lat = _latent(heads, 128, 64, 128, 512)
    mem = dict(heads=heads // 2, dim=128, vdim=2 * 128, gate_cap=15.0)
    return [_layer("latent_attention", **moe, **lat)
            if mix == "latent" or i % 2 == 0
            else _layer("mlstm", **moe, **mem) for i in range(n)]


def _garupel(vocab, width, layers, ff, loop=None) -> dict:
    """layers: (type, sizes) pairs, all with a dense feed-forward."""
    return {"architecture": "Garupel", "vocab": vocab, "width": width,
            "norm": {"eps": 1e-6}, "loop": loop,
            "layers": [{"type": t, "mixer": m,
                        "mlp": {"kind": "dense", "ff": ff} if ff else None}
                       for t, m in layers]}


def _grouped(heads, kv_heads, dim, vdim=None) -> tuple:
    return "attention", dict(heads=heads, kv_heads=kv_heads, dim=dim,
                             vdim=vdim or dim, scale=dim ** -0.5,
                             q_temp={"coef": 0.1, "every": 2048})


def _decays(heads) -> list:
    """1 - 2**(-3 .. -8), evenly over the heads."""
    return [1.0 - 2.0 ** (-3.0 - 5.0 * h / max(heads - 1, 1))
            for h in range(heads)]


def _recurrent_stack(n, width, heads) -> list:
    """Attention, two gated recurrences, linear attention, and so on."""
    kinds = [_grouped(heads, heads // 4, 128),
             ("rglru", dict(width=width, blocks=heads, conv=4)),
             ("rglru", dict(width=width, blocks=heads, conv=4)),
             ("lightning", dict(heads=heads, dim=128, vdim=128,
                                decay=_decays(heads)))]
    return [kinds[i % 4] for i in range(n)]


def _fidizen(vocab, width, layers, taps=4, scale=1.0) -> dict:
    return {"architecture": "Fidizen", "vocab": vocab, "width": width,
            "norm": {"eps": 1e-6}, "embedding": {"scale": scale},
            "canon": {"taps": taps}, "layers": layers}


def _windowed(mlp, heads, dim, rot, vdim, rank, q_rank, window,
              of=None) -> dict:
    mix = {**_latent(heads, dim, rot, vdim, rank), "q_rank": q_rank,
           "mask": {"size": window}}
    d = {"type": "latent_attention", "mixer": mix, "mlp": mlp}
    return d if of is None else {**d, "weights_of": of}


def _poly(ff) -> dict:
    return {"kind": "dense", "ff": ff}


def _sigmoid_moe(experts, top, ff, shared) -> dict:
    return {"kind": "moe", "router": {"experts": experts, "top": top},
            "expert": {"ff": ff}, "shared": {"ff": shared} if shared else None}


def _windowed_stack(n, heads, ff) -> list:
    """Dense and routed layers in turn; two matrices of a dense one are as
    large as the three of the experts that a token uses."""
    mlps = [_poly(9 * ff // 2), _sigmoid_moe(8, 2, ff, ff)]
    return [_windowed(mlps[i % 2], heads, 128, 64, 128, 512, 1024, 1024)
            for i in range(n)]


def _pair(heads, kv_heads, dim, width, chunk, bias_max) -> tuple:
    return "parallel", {
        "left": dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim,
                     scale=dim ** -0.5, bias_max=bias_max,
                     mask={"size": chunk}),
        "right": {"width": width}}


def _ssd(heads, vdim, state, groups, norm_groups=1, conv=4) -> tuple:
    return "mamba2", dict(heads=heads, vdim=vdim, state=state, groups=groups,
                          conv=conv, norm_groups=norm_groups)


def _dogalorn(vocab, width, layers, ff, streams=2, share=(), buckets=65521,
              logit_scale=1.0) -> dict:
    """layers: (type, sizes) pairs; share: owners of further layers."""
    entries = [{"type": t, "mixer": m, "mlp": {"kind": "dense", "ff": ff}}
               for t, m in layers]
    entries += [{**entries[j], "weights_of": j} for j in share]
    return {"architecture": "Dogalorn", "vocab": vocab, "width": width,
            "norm": {"eps": 1e-6}, "streams": streams,
            "logit_scale": logit_scale, "layers": entries,
            "embedding": {"bigram": {"buckets": buckets, "mul_prev": 31,
                                     "mul_cur": 7919}}}


def _paired_stack(n, heads, width) -> list:
    """Pairs of attention and recurrence, and state-space layers, in turn."""
    kinds = [_pair(heads, heads // 4, 128, width, 1024, 128),
             _ssd(width // 32, 64, 128, 1)]
    return [kinds[i % 2] for i in range(n)]


LAYERED_PRESETS = {
    "tiny-dogalorn": _dogalorn(
        336, 72, [_pair(6, 3, 20, 108, 40, 30), _ssd(6, 20, 24, 2, 3),
                  _pair(4, 4, 28, 60, 70, 50)], 104, streams=3, share=(0, 1),
        buckets=500, logit_scale=0.5),
    "dogalorn-2k": _dogalorn(32000, 2048, _paired_stack(8, 16, 2048), 8192),
    "dogalorn-4k": _dogalorn(32000, 4096, _paired_stack(4, 32, 4096), 16384),

    "tiny-fidizen": _fidizen(
        352, 72,
        [_windowed(_poly(104), 5, 20, 12, 28, 44, 36, 70),
         _windowed(_sigmoid_moe(6, 2, 40, 24), 3, 28, 16, 20, 60, 52, 33),
         _windowed(_poly(104), 5, 20, 12, 28, 44, 36, 70, of=0)],
        taps=4, scale=2.0),
    "fidizen-2k": _fidizen(32000, 2048, _windowed_stack(8, 16, 2048)),
    "fidizen-4k": _fidizen(32000, 4096, _windowed_stack(4, 32, 4096)),

    "tiny-garupel": _garupel(
        320, 80,
        [_grouped(6, 3, 20, 28),
         ("rglru", dict(width=108, blocks=3, conv=4)),
         ("lightning", dict(heads=3, dim=24, vdim=40, decay=_decays(3))),
         _grouped(4, 1, 32)], 112,
        loop={"start": 1, "stop": 3, "times": 2}),
    "garupel-2k": _garupel(32000, 2048, _recurrent_stack(8, 2048, 16), 8192),
    "garupel-4k": _garupel(32000, 4096, _recurrent_stack(4, 4096, 32), 16384),

    "tiny-turudra": _design(
        384, 96,
        [_layer("latent_attention", 4, 2, 64, 48, 1.5,
                **_latent(3, 24, 16, 40, 56)),
         _layer("mlstm", 4, 2, 64, 48, 1.5, heads=2, dim=40, vdim=72,
                gate_cap=12.0),
         _layer("latent_attention", 4, 2, 64, 48, 1.5,
                **_latent(3, 24, 16, 40, 56))],
        loop={"start": 0, "stop": 2, "times": 2}),
    # layers of real models' sizes
    "turudra-2k": _design(
        32000, 2048,
        _moe_stack(8, "both", 2048, 16,
                   dict(experts=8, top=2, ff=2048, shared=2048))),
    "turudra-4k": _design(
        32000, 4096,
        _moe_stack(4, "both", 4096, 32,
                   dict(experts=8, top=2, ff=4096, shared=4096))),
}
