"""Layers of the layer-list designs: how a mixer and a feed-forward sit
around the residual stream.

A block runs over a batch and leaves the residual in eng.x, or, where the
next projection can take the last steps along, an output in eng.y whose
norm and addition are still pending (eng.pend).
"""

from __future__ import annotations

from ..ops import hybrid_ops as hy
from .mixers import (FEED_FORWARDS, FEW, FUSE, MIXERS, DenseFF, InputConv,
                     Packer, RoutedExperts)


class Block:
    experts = None

    def new_cache(self, eng):
        """The cache or state of one run of the layer."""
        return self.mixer.new_cache(eng)


class ParallelBlock(Block):
    """x += m (mixer(h) + experts(h)), h the norm of x; the router's rows
    ride along in the input projection."""

    def __init__(self, eng, spec, pk: Packer, i: int):
        p = f"l{i}."
        self.mixer = MIXERS[spec.mixer.kind](eng, spec.mixer, pk, p + "mix.")
        names = [p + "mix." + n for n in self.mixer.IN]
        self.orouter = sum(pk.w[n].shape[0] for n in names)
        self.experts = None
        if spec.mlp:
            names.append(p + "mlp.router")
            self.experts = RoutedExperts(eng, spec.mlp, pk, p + "mlp.")
        self.win = pk.rows(names, eng.W)
        self.ldp = self.p_floats = self.win.shape[0]
        self.act_floats = (self.experts.K1 * self.experts.ffm
                           if self.experts else 0)
        self.g = pk.f32(p + "norm1")

    def run(self, eng, b, cache):
        T, m, ex = b.T, self.mixer, self.experts
        mult = eng.cfg.residual_mult
        few = b.nseg == 0 and T <= FEW
        fuse = few and T <= FUSE
        # norm + every input projection (the router's too)
        eng.project(self.win, eng.h, eng.P, T, self.g)
        if few:
            m.few(eng, b, cache, self, fuse)
        else:
            m.many(eng, b, cache, self)
        if fuse:           # output projection + experts' down + residual
            hy.block_out(eng.f32, m.wo, eng.o, m.ldo,
                         ex.bind(eng) if ex else hy.MoeArgs(),
                         ex.K1 if ex else 0, eng.x, T, eng.W, mult)
        else:
            hy.gemm_rows(eng.o, m.wo, eng.x, T, m.ldo, eng.W, hy.EPI_RESADD,
                         mult=mult)
            if ex:
                ex.many(eng, T, eng.x, mult)


class SandwichBlock(Block):
    """x += norm1b(mixer(norm1(x))), x += norm2b(ff(norm2(x))).  Each post
    norm and addition happens in the staging of the projection after it."""

    def __init__(self, eng, spec, pk: Packer, i: int):
        p = f"l{i}."
        self.mixer = m = MIXERS[spec.mixer.kind](eng, spec.mixer, pk,
                                                 p + "mix.")
        self.win = pk.rows([p + "mix." + n for n in m.IN], eng.W)
        self.bias = m.biases(pk, p + "mix.")
        self.ldp = self.p_floats = self.win.shape[0]
        self.g1, self.g1b = pk.f32(p + "norm1"), pk.f32(p + "norm1b")
        self.ff = None
        self.act_floats = 0
        if spec.mlp:
            self.ff = DenseFF(eng, spec.mlp, pk, p + "mlp.")
            self.act_floats = self.ff.ffp
            self.g2, self.g2b = pk.f32(p + "norm2"), pk.f32(p + "norm2b")

    def run(self, eng, b, cache):
        T = b.T
        eng.project(self.win, eng.h, eng.P, T, self.g1, bias=self.bias)
        self.mixer.run(eng, b, cache, self)
        self.mixer.out(eng, b, self)
        eng.pend = self.g1b
        if self.ff:
            eng.project(self.ff.up, eng.h, eng.act, T, self.g2,
                        epi=hy.EPI_RELU2)
            eng.linear(self.ff.down, eng.act, eng.y, T)
            eng.pend = self.g2b


class PostNormBlock(Block):
    """x += norm1(mixer(c1(x))), x += norm2(ff(c2(x))), c a short causal
    convolution over time added to its input.  Norm and addition happen in
    the staging of the projection after them, together with its
    convolution."""

    def __init__(self, eng, spec, pk: Packer, i: int):
        p = f"l{i}."
        self.mixer = m = MIXERS[spec.mixer.kind](eng, spec.mixer, pk,
                                                 p + "mix.")
        self.win = pk.rows([p + "mix." + n for n in m.IN], eng.W)
        self.ldp = self.p_floats = self.win.shape[0]
        self.orouter = self.act_floats = 0
        self.c1, self.g1 = InputConv(pk, p + "canon1"), pk.f32(p + "norm1")
        self.ff = None
        if spec.mlp:
            self.ff = FEED_FORWARDS[spec.mlp.kind](eng, spec.mlp, pk,
                                                   p + "mlp.")
            self.c2, self.g2 = InputConv(pk, p + "canon2"), pk.f32(p + "norm2")
            self.act_floats = self.ff.act_floats
            self.p_floats = max(self.ldp, self.ff.p_floats)

    def new_cache(self, eng):
        convs = [self.c1, self.c2] if self.ff else [self.c1]
        return (self.mixer.new_cache(eng), *(c.new_ring(eng) for c in convs))

    def run(self, eng, b, cache):
        eng.conv_project(self.win, self.c1.w, cache[1], b, eng.P)
        self.mixer.run(eng, b, cache[0], self)
        self.mixer.out(eng, b, self)
        eng.pend = self.g1
        if self.ff:
            across = eng.conv_project(self.ff.up, self.c2.w, cache[2], b,
                                      eng.P, self.ff.experts is not None)
            self.ff.after_up(eng, b, across)
            eng.pend = self.g2


class HyperMix:
    """How a sublayer reads the residual streams (read), and how they all
    turn (mix [from, to]) and take up its output (feed)."""

    def __init__(self, pk: Packer, p: str):
        self.read, self.feed = pk.f32(p + "in"), pk.f32(p + "out")
        self.mix = pk.f32(p + "mix")


class HyperBlock(Block):
    """x_t <- sum_s mix[s, t] x_s + feed[t] f(norm(sum_s read[s] x_s)) for
    mixer and feed-forward f.  The streams turn in the staging of the
    projection after them."""

    def __init__(self, eng, spec, pk: Packer, i: int):
        p = f"l{i}."
        self.mixer = m = MIXERS[spec.mixer.kind](eng, spec.mixer, pk,
                                                 p + "mix.")
        self.win = pk.rows([p + "mix." + n for n in m.IN], eng.W)
        self.bias = m.biases(pk, p + "mix.")
        self.ldp = self.p_floats = self.win.shape[0]
        self.g1, self.c1 = pk.f32(p + "norm1"), HyperMix(pk, p + "hc1.")
        self.ff = None
        self.act_floats = 0
        if spec.mlp:
            self.ff = FEED_FORWARDS[spec.mlp.kind](eng, spec.mlp, pk,
                                                   p + "mlp.")
            self.act_floats = self.ff.act_floats
            self.g2, self.c2 = pk.f32(p + "norm2"), HyperMix(pk, p + "hc2.")

    def run(self, eng, b, cache):
        T, m, ff = b.T, self.mixer, self.ff
        eng.read_streams(self.win, eng.P, T, self.c1.read, self.g1,
                         bias=self.bias)
        m.run(eng, b, cache, self)
        m.out(eng, b, self)
        eng.turn = (self.c1, m.halves(eng) if hasattr(m, "halves") else {})
        if ff:
            eng.read_streams(ff.up, eng.act, T, self.c2.read, self.g2,
                             bias=ff.bias, epi=hy.EPI_GELU)
            eng.linear(ff.down, eng.act, eng.y, T, bias=ff.down_bias)
            eng.turn = (self.c2, {})


BLOCKS = {"parallel": ParallelBlock, "sandwich": SandwichBlock,
          "post": PostNormBlock, "hyper": HyperBlock}
