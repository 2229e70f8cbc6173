"""Device side of the layer-list mechanisms: weights in kernel layout, the
cache or state of each layer run, and the kernel sequence for a batch.

Every mechanism has two sequences over the same cache and state:

    few()   up to 16 rows, one token each (decode): fused small launches;
            with `fuse` the experts' gate/up halves ride along
    many()  any mix of single tokens and runs of tokens: MFMA GEMMs, run
            kernels over the runs, single-token kernels over the rest

A batch lists its single-token rows first.  Both leave the mixer's output
(before the output projection) in eng.o and, in a parallel block, the
expert choice in eng.ridx / eng.rwt.  Mixers of sandwich and post blocks
have run(), which picks the sequence, and apply their output projection
themselves, in out().
"""

from __future__ import annotations

import numpy as np
import torch

from ..ops import hybrid_ops as hy

PART_FLOATS = 1 << 25     # split-attention scratch for prompt portions
FEW = 16            # single tokens that take the fused few-row kernels
FUSE = 5            # of them, those whose experts run as fused GEMVs


def pad_to(n: int, m: int) -> int:
    return -(-n // m) * m


class Packer:
    """Checkpoint arrays -> device tensors in kernel layout."""

    def __init__(self, weights, device, dtype):
        self.w, self.device, self.dtype = weights, device, dtype

    def raw(self, name) -> torch.Tensor:
        return torch.from_numpy(self.w[name]).to(self.device)

    def f32(self, name) -> torch.Tensor:
        return self.raw(name).float().contiguous()

    def rows(self, names, K: int) -> torch.Tensor:
        """[sum of rows, K padded to 64] of [rows, K] matrices."""
        mats = [self.raw(n) for n in names]
        out = torch.zeros(sum(m.shape[0] for m in mats), pad_to(K, 64),
                          dtype=self.dtype, device=self.device)
        r = 0
        for m in mats:
            out[r:r + m.shape[0], :K].copy_(m)
            r += m.shape[0]
        return out


class RoutedExperts:
    """Routed experts and their shared one (see csrc/moe.h for the weight
    layout).  Routing logits are columns of a parallel block's input
    projection, so the router costs no launch of its own there; elsewhere
    they are a projection by themselves."""

    def __init__(self, eng, spec, pk: Packer, p: str):
        W, Wp = eng.W, eng.Wp
        E, sh = spec.experts, spec.shared
        self.spec, self.top, self.extra = spec, spec.top, 1 if sh else 0
        self.K1 = self.top + self.extra
        ff = self.ff = pad_to(spec.expert.ff, 64)
        ffs = self.ffs = pad_to(sh.ff, 64) if sh else ff
        self.ffm = max(ff, ffs) if sh else ff
        kw = dict(dtype=pk.dtype, device=pk.device)
        self.gu = torch.zeros((E * ff + (ffs if sh else 0)) * 2 * Wp, **kw)
        self.down = torch.zeros((E * ff + (ffs if sh else 0)) * W, **kw)

        def fill(q, e, n, fp):
            gu = self.gu[e * ff * 2 * Wp:][:2 * fp * Wp].view(
                fp // 16, 2, 16, Wp)
            for half, name in ((0, "gate"), (1, "up")):
                full = torch.zeros(fp, Wp, **kw)
                full[:n, :W].copy_(pk.raw(q + name))
                gu[:, half].copy_(full.view(fp // 16, 16, Wp))
            self.down[e * ff * W:][:W * fp].view(W, fp)[:, :n].copy_(
                pk.raw(q + "down"))

        for e in range(E):
            fill(f"{p}e{e}.", e, spec.expert.ff, ff)
        if sh:
            fill(p + "shared.", E, sh.ff, ffs)
        self.args = hy.MoeArgs().put(
            gu=self.gu, down=self.down, ldh=Wp, ldact=self.ffm, W=W, E=E,
            K1=self.K1, ff=ff, ffs=ffs, glu=int(spec.glu == "silu"),
            win=int(spec.weigh == "input"), lim=spec.expert.limit,
            lims=sh.limit if sh else 0.0)

    def bind(self, eng):
        return self.args.put(h=eng.h, idx=eng.ridx, wt=eng.rwt, act=eng.act)

    def route(self, eng, T: int, across: bool):
        """Routing of the logits in eng.P, [T, E] or (across) [E, T]."""
        E = self.spec.experts
        return hy.RouteArgs().put(
            z=eng.P, idx=eng.ridx, wt=eng.rwt, ldz=1 if across else E,
            lde=T if across else 1, rows=T, E=E,
            top=self.top, extra=self.extra,
            scores=int(self.spec.score == "sigmoid"))

    def apart(self, eng, T: int, few: bool, across: bool):
        """eng.y = the experts' sum for the rows of eng.h, from the logits
        in eng.P."""
        m, route = self.bind(eng), self.route(eng, T, across)
        if few and T <= FUSE:
            hy.moe_gu_few(eng.f32, m, route)
            hy.block_out(eng.f32, None, None, 0, m, self.K1, eng.y, T, eng.W,
                         1.0, set=True)
        else:
            hy.moe_route(m, route)
            self.many(eng, T, eng.y, 1.0, True)

    def many(self, eng, T: int, out, mult: float, set: bool = False):
        avg = T * self.top / self.spec.experts
        bm = 128 if avg >= 160 else 64 if avg >= 24 else 32
        pairs, groups = T * self.K1, self.spec.experts + self.extra
        s = hy.MoeSort().put(
            perm=eng.perm, tile_e=eng.tile_e, tile_row0=eng.tile_row0,
            tile_n=eng.tile_n, pairs=pairs, groups=groups, bm=bm,
            maxtiles=pairs // bm + groups)
        assert s.maxtiles <= eng.tile_e.numel()
        hy.moe_rows(eng.f32, self.bind(eng), s, eng.ypair, out, T, mult, set)


class LatentAttention:
    kind = "latent_attention"

    def __init__(self, eng, spec, pk: Packer, p: str):
        self.spec = s = spec
        fit = [r for r in hy.RANKS if r >= s.kv_rank]
        if not fit or s.rot_dim > 128:
            raise ValueError(
                f"latent attention: kv_rank {s.kv_rank} / rot_dim "
                f"{s.rot_dim} exceed the built kernels "
                f"({hy.RANKS[-1]} / 128)")
        self.IN = s.inputs                 # rows of the input projection
        self.RP, self.RT = fit[0], pad_to(s.rot_dim, 32)
        self.tile_pairs = s.heads          # pairs a token adds to a tile
        self.CS, self.dp = self.RP + self.RT, pad_to(s.dim, 64)
        H, d, vd, RP = s.heads, s.dim, s.vdim, self.RP
        kw = dict(dtype=pk.dtype, device=pk.device)
        uk = pk.raw(p + "uk").view(H, d, s.kv_rank)
        self.wuk = torch.zeros(H, d, RP, **kw)
        self.wuk[:, :, :s.kv_rank].copy_(uk)
        self.wukT = torch.zeros(H, RP, self.dp, **kw)
        self.wukT[:, :s.kv_rank, :d].copy_(uk.transpose(1, 2))
        self.wuv = torch.zeros(H, vd, RP, **kw)
        self.wuv[:, :, :s.kv_rank].copy_(
            pk.raw(p + "uv").view(H, vd, s.kv_rank))
        self.ldo = pad_to(H * vd, 64)
        self.wo = pk.rows([p + "o"], H * vd)
        self.cnorm = pk.f32(p + "dkv.norm")
        self.cosT, self.sinT = eng.rope_tables(s.rot_base, s.rot_dims)
        nq = s.q_rank or H * (d + s.rot_dim)
        self.og = nq + s.kv_rank + s.rot_dim
        each = s.gate == "element"
        self.args = hy.LatentArgs().put(
            Wuk=self.wuk, Wuv=self.wuv, cnorm=self.cnorm, cosT=self.cosT,
            sinT=self.sinT, oq=0, odkv=nq, og=self.og, H=H, d=d, dp=self.dp,
            rot=s.rot_dim, rdims=s.rot_dims, RT=self.RT, rank=s.kv_rank,
            RP=RP, vd=vd, ldo=self.ldo, qh=d + s.rot_dim, oqr=d,
            qrh=d + s.rot_dim, pairs=int(s.interleaved), win=s.window or 0,
            gz=vd if each else 1, gc=int(each), eps=eng.cfg.norm_eps,
            scale=s.scale)
        if s.sink:
            self.sink = pk.f32(p + "sink")
            self.args.put(sink=self.sink)
        if s.q_rank:
            self._query_latent(pk, p)

    def _query_latent(self, pk: Packer, p: str):
        """W_uq with the unrotated parts of all heads first, each padded to
        dp rows, then the rotated ones, each padded to RT."""
        s, H, dp, RT = self.spec, self.spec.heads, self.dp, self.RT
        uq = pk.rows([p + "uq"], s.q_rank)
        self.QRp = uq.shape[1]
        uq = uq.view(H, s.dim + s.rot_dim, self.QRp)
        self.wuq = torch.zeros(H * (dp + RT), self.QRp, dtype=pk.dtype,
                               device=pk.device)
        flat, rot = self.wuq[:H * dp], self.wuq[H * dp:]
        flat.view(H, dp, -1)[:, :s.dim].copy_(uq[:, :s.dim])
        rot.view(H, RT, -1)[:, :s.rot_dim].copy_(uq[:, s.dim:])
        self.qnorm = pk.f32(p + "dq.norm")
        self.args.put(qnorm=self.qnorm, qrank=s.q_rank, QRp=self.QRp,
                      ldq=H * (dp + RT), qh=dp, oqr=H * dp, qrh=RT)

    def new_cache(self, eng):
        return torch.zeros(eng.cache.num_pages, hy.PAGE, self.CS,
                           dtype=eng.T, device=eng.device)

    def token_splits(self, eng, rows: int) -> int:
        """Key splits of single tokens, at most one per key tile of the
        window."""
        n = eng.decode_splits(rows)
        return max(2, min(n, self.spec.window // 32 + 1)) \
            if self.spec.window else n

    def sizes(self, eng, rows):
        """Scratch elements for `rows` rows, and fp32 partials."""
        H = self.spec.heads
        splits = max(PART_FLOATS // (H * self.RP),
                     *(r * eng.decode_splits(r)
                       for r in range(1, eng.max_batch + 1)), 1)
        need = dict(qn=rows * H * self.dp, qa=rows * H * self.CS,
                    olat=rows * H * self.RP, o=rows * self.ldo,
                    part=splits * H * self.RP, ml=splits * H * 2)
        if self.spec.q_rank:
            need.update(cq=rows * self.QRp,
                        qf=min(rows, FEW) * self.wuq.shape[0])
        return need

    def _bind(self, eng, b, cache, layer):
        x, latent = layer.experts, self.spec.q_rank
        if not latent:
            self.args.put(ldq=layer.ldp)
        return self.args.put(
            P=eng.P, Q=eng.qf if latent else eng.P, cq=eng.cq, slot=b.slot,
            pos=b.pos, table=eng.table, cache=cache, qn=eng.qn, qa=eng.qa,
            part=eng.part, ml=eng.ml, olat=eng.olat, o=eng.o,
            seg_row0=b.seg_row0, seg_len=b.seg_len, seg_slot=b.seg_slot,
            seg_pos0=b.seg_pos0, tile_seg=0, tile_rr0=0, ridx=eng.ridx,
            rwt=eng.rwt, ldp=layer.ldp, orouter=layer.orouter,
            ldt=eng.table.shape[1], rows=b.T, rbase=0, NS=1, written=0,
            E=x.spec.experts if x else 0, rtop=x.top if x else 0,
            rextra=x.extra if x else 0)

    def _single(self, eng, a, n):
        """Split attention of the first n rows, partials left in part/ml."""
        a.put(rows=n, rbase=0, NS=self.token_splits(eng, n))
        hy.latent_attn(eng.f32, a, 1, n * (-(-self.spec.heads // 16)))

    def _queries(self, eng, a, T):
        """Queries of a few rows, fp32, from their latents."""
        s = self.spec
        if eng.one_row(self.wuq, T):
            hy.lin_row(self.wuq, eng.P, eng.qf, s.q_rank, eng.cfg.norm_eps,
                       g=self.qnorm)
        else:
            hy.latent_mid(eng.f32, a)
            a.put(written=1)
            hy.gemm_rows(eng.cq, self.wuq, eng.qf, T, self.QRp,
                         self.wuq.shape[0], hy.EPI_F32)

    def few(self, eng, b, cache, layer, fuse):
        a = self._bind(eng, b, cache, layer)
        if self.spec.q_rank:
            self._queries(eng, a, b.T)
        hy.latent_dec_prep(eng.f32, a)
        self._single(eng, a, b.T)
        x = layer.experts if fuse else None
        hy.latent_dec_fin(eng.f32, a, x.bind(eng) if x else hy.MoeArgs(),
                          b.T * x.K1 if x else 0)

    def many(self, eng, b, cache, layer):
        s, H, CS, RP = self.spec, self.spec.heads, self.CS, self.RP
        a = self._bind(eng, b, cache, layer)
        if s.q_rank:
            hy.latent_mid(eng.f32, a)
            rot = hy.Rotary().put(
                pos=b.pos, cosT=self.cosT, sinT=self.sinT, y=eng.qa[RP:],
                split=H * self.dp, RT=self.RT, dims=s.rot_dims, ld=H * CS,
                hs=CS)
            hy.gemm_rows(eng.cq, self.wuq, eng.qn, b.T, self.QRp,
                         H * self.dp, hy.EPI_ROTARY, rotary=rot)
        else:
            hy.latent_prep(eng.f32, a)
        hy.gemm_rows(eng.qn, self.wukT, eng.qa, b.T, H * self.dp, H * CS,
                     hy.EPI_T, N=RP, K=self.dp, Z=H, xz=self.dp,
                     wz=RP * self.dp, yz=CS)
        if b.nd:
            self._single(eng, a, b.nd)
            hy.latent_merge(eng.f32, a)
        if b.nd < b.T:
            seg, rr0, n, longest = b.tiles[H]
            if s.window:
                longest = min(longest, s.window + hy.TILE // H)
            rows = b.T - b.nd
            ns = min(eng.run_splits(n, longest),
                     eng.part.numel() // (rows * H * RP),
                     eng.ml.numel() // (rows * H * 2))
            a.put(tile_seg=seg, tile_rr0=rr0, rows=rows, rbase=b.nd,
                  NS=max(1, ns))
            hy.latent_attn(eng.f32, a, 0, n)
            if ns > 1:
                hy.latent_merge(eng.f32, a)
        hy.gemm_rows(eng.olat, self.wuv, eng.o, b.T, H * RP, self.ldo,
                     hy.EPI_TGATE, N=s.vdim, K=RP, Z=H, xz=RP,
                     wz=s.vdim * RP, yz=s.vdim, gate=eng.P[self.og:],
                     ldg=layer.ldp, gz=a.gz, gc=a.gc)

    def run(self, eng, b, cache, layer):
        if b.nseg == 0 and b.T <= FEW:
            self.few(eng, b, cache, layer, False)
        else:
            self.many(eng, b, cache, layer)

    def out(self, eng, b, layer):
        eng.linear(self.wo, eng.o, eng.y, b.T)


class MLSTM:
    kind = "mlstm"
    tile_pairs = None
    IN = ("q", "k", "v", "g", "i", "f")

    def __init__(self, eng, spec, pk: Packer, p: str):
        self.spec = s = spec
        H, d, vd = s.heads, s.dim, s.vdim
        if d > 8192:
            raise ValueError(f"mlstm: dim {d} exceeds the built kernels")
        self.nvt = -(-vd // 64)
        self.ldo = pad_to(H * vd, 64)
        self.wo = pk.rows([p + "o"], H * vd)
        self.ib, self.fb = pk.f32(p + "i.b"), pk.f32(p + "f.b")
        self.norm = pk.f32(p + "norm")
        qk, v = H * d, H * vd
        self.args = hy.MlstmArgs().put(
            ib=self.ib, fb=self.fb, norm=self.norm, oq=0, ok=qk, ov=2 * qk,
            og=2 * qk + v, oi=2 * qk + 2 * v, of=2 * qk + 2 * v + H, H=H, d=d,
            vd=vd, nvt=self.nvt, ldo=self.ldo, cap=s.gate_cap,
            eps=eng.cfg.norm_eps)

    def new_cache(self, eng):
        n, s = eng.cache.num_slots, self.spec
        z = lambda *sh: torch.zeros(*sh, dtype=torch.float32,
                                    device=eng.device)
        return (z(n, s.heads, s.dim, s.vdim), z(n, s.heads, self.nvt, s.dim),
                z(n, s.heads, self.nvt))

    def sizes(self, eng, rows):
        s, chunks = self.spec, eng.max_chunks(rows)
        return dict(o=rows * self.ldo, raw=rows * s.heads * s.vdim,
                    gF=rows * s.heads, gi=rows * s.heads, gm=rows * s.heads,
                    cm0=chunks * s.heads,
                    U=chunks * s.heads * s.dim * s.vdim,
                    un=chunks * s.heads * s.dim)

    def _bind(self, eng, b, cache, layer):
        x, nd = layer.experts, b.nd
        S, n, m = cache
        return self.args.put(
            P=eng.P, S=S, n=n, m=m, o=eng.raw, out=eng.o, slot=b.slot,
            pos=b.pos, seg_row0=b.seg_row0[nd:], seg_len=b.seg_len[nd:],
            seg_slot=b.seg_slot[nd:], seg_pos0=b.seg_pos0[nd:],
            seg_chunk0=b.seg_chunk0, chunk_row0=b.chunk_row0,
            chunk_len=b.chunk_len, gF=eng.gF, gi=eng.gi, gm=eng.gm,
            cm0=eng.cm0, U=eng.U, un=eng.un, ridx=eng.ridx, rwt=eng.rwt,
            ldp=layer.ldp, orouter=layer.orouter, rows=b.T, nseg=b.nseg,
            nchunk=b.nchunk, E=x.spec.experts if x else 0,
            rtop=x.top if x else 0, rextra=x.extra if x else 0)

    def few(self, eng, b, cache, layer, fuse):
        a = self._bind(eng, b, cache, layer)
        x = layer.experts if fuse else None
        hy.mlstm_step(a)
        hy.mlstm_dec_fin(eng.f32, a, x.bind(eng) if x else hy.MoeArgs(),
                         b.T * x.K1 if x else 0)

    def many(self, eng, b, cache, layer):
        a = self._bind(eng, b, cache, layer)
        if b.nd:
            E = a.E
            hy.mlstm_step(a.put(rows=b.nd, E=0))
            a.put(rows=b.T, E=E)
        if b.nseg:
            hy.mlstm_chunks(a)
        hy.mlstm_post(eng.f32, a)


class SandwichMixer:
    """A mixer whose batch has one kernel sequence; the projections named in
    IN run as one matrix, with the biases of those that have one."""
    tile_pairs = None

    def biases(self, pk: Packer, p: str):
        parts = [pk.f32(p + n + ".b") if p + n + ".b" in pk.w else
                 torch.zeros(pk.w[p + n].shape[0], device=pk.device)
                 for n in self.IN]
        return (torch.cat(parts) if any(p + n + ".b" in pk.w
                                        for n in self.IN) else None)

    def out(self, eng, b, layer):
        """eng.y = W_o . the mixer's output."""
        eng.linear(self.wo, eng.o, eng.y, b.T)


def distance_bias(rel: np.ndarray, far: float, longest: int) -> np.ndarray:
    """[heads, n] bias by distance from the buckets rel [rows, heads]: below
    rows/2 a bucket per distance, then logarithmic up to `far`.  Every
    distance from n - 1 on has the last value."""
    rows, half = len(rel), len(rel) // 2
    if rows < 2 or rows % 2 or far <= half:
        raise ValueError(f"attention: {rows} bias buckets up to distance "
                         f"{far} are not possible")
    n = np.arange(min(longest, int(np.ceil(far)) + 1))
    log = half + np.floor(np.log(np.maximum(n, half) / half) /
                          np.log(far / half) * (rows - half))
    return rel[np.where(n < half, n, np.minimum(rows - 1, log)).astype(int)].T


class GroupedAttention(SandwichMixer):
    kind = "attention"

    def __init__(self, eng, spec, pk: Packer, p: str):
        self.spec = s = spec
        self.IN = s.inputs
        fit = [c for c in hy.HEAD_SIZES if c[0] >= s.dim and c[1] >= s.vdim]
        if not fit:
            raise ValueError(
                f"attention: head sizes {s.dim}/{s.vdim} exceed the built "
                f"kernels ({hy.HEAD_SIZES[-1]})")
        self.DP, self.VP = fit[0]
        H, G = s.heads, s.kv_heads
        self.tile_pairs = H // G
        self.ldo = pad_to(H * s.vdim, 64)
        self.wo = pk.rows([p + "o"], H * s.vdim)
        self.qnorm, self.knorm = pk.f32(p + "q.norm"), pk.f32(p + "k.norm")
        q, k, v = H * s.dim, G * s.dim, G * s.vdim
        own = "v" in s.inputs                 # else the values are the keys
        self.args = hy.GqaArgs().put(
            qnorm=self.qnorm, knorm=self.knorm, oq=0, ok=q,
            ov=q + k if own else q, og=q + k + v if "g" in s.inputs else -1,
            H=H, G=G, d=s.dim, vd=s.vdim,
            DP=self.DP, VP=self.VP, ldo=self.ldo, eps=eng.cfg.norm_eps,
            scale=s.scale, chunk=min(s.chunk or 0, eng.max_seq))
        if s.bias_max is None:
            self.temp = eng.query_temperature(s.temp_coef, s.temp_every)
            self.args.put(temp=self.temp)
        else:
            self._biases(eng, pk, p)
        if s.sink:
            self.sink = torch.zeros(H, device=pk.device)
            self.args.put(sink=self.sink)

    def _biases(self, eng, pk: Packer, p: str):
        """Distance biases, base 2, and the numbers per head folded into the
        norm of the queries."""
        s = self.spec
        longest = min(s.chunk or eng.max_seq, eng.max_seq)
        rel = distance_bias(np.asarray(pk.w[p + "rel"], np.float64),
                            s.bias_max, longest)
        room = (30 if self.DP == 256 else 90) * 1024
        if self.tile_pairs * rel.shape[1] * 4 > room:
            raise ValueError(
                f"attention: {rel.shape[1]} distances for {self.tile_pairs} "
                f"heads exceed the built kernels")
        self.bias = torch.from_numpy(
            (rel * np.log2(np.e)).astype(np.float32)).to(pk.device).contiguous()
        self.qnorm = (self.qnorm.view(s.heads, s.dim) *
                      pk.f32(p + "temp")[:, None]).contiguous()
        self.args.put(bias=self.bias, nbias=rel.shape[1], qnorm=self.qnorm)

    def new_cache(self, eng):
        n, G = eng.cache.num_pages, self.spec.kv_heads
        kw = dict(dtype=eng.T, device=eng.device)
        return (torch.zeros(n, G, hy.PAGE, self.DP, **kw),
                torch.zeros(n, G, self.VP, hy.PAGE, **kw))

    def token_splits(self, eng, rows: int) -> int:
        """Shares of the keys for single tokens, 128 keys at a time: fixed
        by the cache size and the number of rows, so a captured step keeps
        its grid."""
        groups = -(-eng.cache.table.shape[1] * hy.PAGE // 128)
        if self.spec.chunk:
            groups = min(groups, self.spec.chunk // 128 + 2)
        blocks = rows * self.spec.kv_heads * -(-self.tile_pairs // 16)
        return int(max(1, min(64, groups, 1024 // blocks)))

    def sizes(self, eng, rows):
        H = self.spec.heads
        splits = max(PART_FLOATS // (H * self.VP),
                     *(r * self.token_splits(eng, r)
                       for r in range(1, eng.max_batch + 1)), 1)
        return dict(q=rows * H * self.DP, o=rows * self.ldo,
                    part=splits * H * self.VP, ml=splits * H * 2)

    def run(self, eng, b, cache, layer, beside=None):
        """beside: arguments of a gated recurrence whose single tokens take
        their step along with this one's."""
        s, H, R = self.spec, self.spec.heads, self.tile_pairs
        a = self.args.put(
            P=eng.P, slot=b.slot, pos=b.pos, table=eng.table, K=cache[0],
            V=cache[1], q=eng.q, part=eng.part, ml=eng.ml, o=eng.o,
            seg_row0=b.seg_row0, seg_len=b.seg_len, seg_slot=b.seg_slot,
            seg_pos0=b.seg_pos0, ldp=layer.ldp, ldt=eng.table.shape[1])
        if b.nd:
            a.put(rows=b.nd, rbase=0, NS=self.token_splits(eng, b.nd))
            hy.gqa_token(eng.f32, a)
            hy.gqa_merge(eng.f32, a, beside)
        if b.nd < b.T:
            rows = b.T - b.nd
            seg, rr0, n, longest = b.tiles[R]
            if s.chunk:
                longest = min(longest, s.chunk + hy.TILE // R)
            ns = min(eng.run_splits(n * s.kv_heads, longest),
                     eng.part.numel() // (rows * H * self.VP),
                     eng.ml.numel() // (rows * H * 2))
            a.put(tile_seg=seg, tile_rr0=rr0, rows=rows, rbase=b.nd,
                  NS=max(1, ns))
            hy.gqa_prep(eng.f32, a)
            hy.gqa_run(eng.f32, a, n)
            if ns > 1:
                hy.gqa_merge(eng.f32, a)


class MinGRU(SandwichMixer):
    kind = "mingru"

    def __init__(self, eng, spec, pk: Packer, p: str):
        self.spec, self.IN, C = spec, spec.inputs, spec.width
        self.ldo = pad_to(C, 64)
        self.wo = pk.rows([p + "o"], C)
        self.args = hy.MingruArgs().put(oz=0, ox=C, og=2 * C, C=C,
                                        ldo=self.ldo)

    def new_cache(self, eng):
        return (torch.zeros(eng.cache.num_slots, self.spec.width,
                            dtype=torch.float32, device=eng.device),)

    def sizes(self, eng, rows):
        n = eng.max_chunks(rows) * self.spec.width
        return dict(o=rows * self.ldo, decay=n, local=n)

    def bind(self, eng, b, cache, layer):
        nd = b.nd
        return self.args.put(
            P=eng.P, S=cache[0], A=eng.decay, h=eng.local, out=eng.o,
            slot=b.slot, pos=b.pos, seg_row0=b.seg_row0[nd:],
            seg_len=b.seg_len[nd:], seg_slot=b.seg_slot[nd:],
            seg_pos0=b.seg_pos0[nd:], chunk_row0=b.chunk_row0,
            chunk_len=b.chunk_len, chunk_seg=b.chunk_seg, ldp=layer.ldp,
            rows=nd, nchunk=b.nchunk)

    def run(self, eng, b, cache, layer):
        a = self.bind(eng, b, cache, layer)
        if b.nd:
            hy.mingru_step(eng.f32, a)
        if b.nseg:
            hy.mingru_run(eng.f32, a)


class MixerPair(SandwichMixer):
    """Attention and a gated recurrence side by side: one input projection,
    their outputs beside each other in eng.o, one launch for both output
    projections into the halves of eng.y.  The norms of the halves and their
    sum are left to the staging of the next projection."""
    kind = "parallel"

    def __init__(self, eng, spec, pk: Packer, p: str):
        self.spec = spec
        l, r = self.parts = [
            MIXERS[s.kind](eng, s, pk, f"{p}{k}.")
            for k, s in (("left", spec.left), ("right", spec.right))]
        self.IN = tuple(f"{k}.{n}" for k, m in (("left", l), ("right", r))
                        for n in m.IN)
        self.tile_pairs = l.tile_pairs
        at = sum(pk.w[f"{p}left.{n}"].shape[0] for n in l.IN)
        self.ldo = l.ldo + r.ldo
        l.args.put(ldo=self.ldo)
        r.args.put(ldo=self.ldo, **{o: getattr(r.args, o) + at
                                    for o in ("oz", "ox", "og")})
        self.wo = torch.cat([m.wo.flatten() for m in (l, r)])
        self.W = l.wo.shape[0]
        self.wl = self.wo[:l.wo.numel()].view_as(l.wo)
        l.wo = r.wo = None
        self.gl, self.gr = pk.f32(p + "left.out"), pk.f32(p + "right.out")

    def new_cache(self, eng):
        return tuple(m.new_cache(eng) for m in self.parts)

    def sizes(self, eng, rows):
        a, b = (m.sizes(eng, rows) for m in self.parts)
        return {**{k: max(a.get(k, 0), b.get(k, 0)) for k in {*a, *b}},
                "o": rows * self.ldo}

    def run(self, eng, b, cache, layer):
        l, r = self.parts
        a = r.bind(eng, b, cache[1], layer).put(out=eng.o[l.ldo:])
        l.run(eng, b, cache[0], layer, beside=a)
        if b.nseg:
            hy.mingru_run(eng.f32, a)

    def out(self, eng, b, layer):
        l, r = self.parts
        W, T, half = self.W, b.T, eng.PC * self.W
        if eng.one_row(self.wl, T):
            hy.lin_row(self.wl, None, eng.y, 0, 0.0, hin=eng.o,
                       second=(r.ldo, l.ldo, W * l.ldo, half))
        else:
            hy.gemm_rows(eng.o, self.wo, eng.y, T, self.ldo, W, hy.EPI_F32,
                         N=W, K=l.ldo, Z=2, xz=l.ldo, wz=W * l.ldo, yz=half,
                         K2=r.ldo)

    def halves(self, eng):
        """How the staging after it puts the output together."""
        return dict(y2=eng.y[1], gb=self.gl, gb2=self.gr)


class SSD(SandwichMixer):
    kind = "mamba2"

    def __init__(self, eng, spec, pk: Packer, p: str):
        self.spec, self.IN = spec, spec.inputs
        s = spec
        if s.state > 8192 or s.norm_groups > hy.MAX_GROUPS:
            raise ValueError(f"mamba2: state {s.state} or norm_groups "
                             f"{s.norm_groups} exceed the built kernels")
        self.ldo = pad_to(s.inner, 64)
        self.wo = pk.rows([p + "o"], s.inner)
        self.norm = pk.f32(p + "norm")
        self.cw = pk.f32(p + "conv").t().contiguous()
        self.cb, self.dtb = pk.f32(p + "conv.b"), pk.f32(p + "dt_bias")
        self.rate = torch.from_numpy(-np.exp(np.asarray(
            pk.w[p + "A_log"], np.float64)).astype(np.float32)).to(pk.device)
        self.D = pk.f32(p + "D")
        self.args = hy.SsdArgs().put(
            cw=self.cw, cb=self.cb, dtb=self.dtb, rate=self.rate, D=self.D,
            oz=0, ox=s.inner, odt=s.inner + s.channels, H=s.heads,
            G=s.groups, N=s.state, vd=s.vdim, C=s.channels, taps=s.conv,
            nvt=-(-s.vdim // 64))

    def new_cache(self, eng):
        n, s = eng.cache.num_slots, self.spec
        kw = dict(dtype=torch.float32, device=eng.device)
        return (torch.zeros(n, s.heads, s.state, s.vdim, **kw),
                torch.zeros(n, s.conv, s.channels, **kw))

    def sizes(self, eng, rows):
        s = self.spec
        return dict(o=rows * self.ldo, raw=rows * s.inner,
                    u=rows * s.channels, gi=rows * s.heads,
                    gF=rows * s.heads,
                    U=eng.max_chunks(rows) * s.heads * s.state * s.vdim)

    def run(self, eng, b, cache, layer):
        nd = b.nd
        a = self.args.put(
            P=eng.P, S=cache[0], ring=cache[1], u=eng.u, dt=eng.gi, L=eng.gF,
            U=eng.U, o=eng.raw, slot=b.slot, pos=b.pos,
            seg_row0=b.seg_row0[nd:], seg_len=b.seg_len[nd:],
            seg_slot=b.seg_slot[nd:], seg_pos0=b.seg_pos0[nd:],
            seg_chunk0=b.seg_chunk0, chunk_row0=b.chunk_row0,
            chunk_len=b.chunk_len, chunk_seg=b.chunk_seg, ldp=layer.ldp,
            rows=max(nd, 1), nseg=b.nseg, nchunk=b.nchunk)
        if nd:
            hy.ssd_step(a)
        if b.nseg:
            hy.ssd_run(a)

    def out(self, eng, b, layer):
        """Normed in parts, projected."""
        eng.normed_linear(self.wo, eng.o, eng.y, b.T, eng.raw,
                          self.spec.inner, self.norm,
                          groups=self.spec.norm_groups)


class RGLRU(SandwichMixer):
    kind = "rglru"
    IN = ("y", "x")

    def __init__(self, eng, spec, pk: Packer, p: str):
        self.spec = s = spec
        C, nb = s.width, s.blocks
        bw = C // nb
        KP = pad_to(bw, 64)
        if KP * 4 > 150 * 1024:
            raise ValueError(f"rglru: {bw} channels in a block exceed the "
                             f"built kernels")
        self.ldo = pad_to(C, 64)
        self.wo = pk.rows([p + "o"], C)
        self.gates = torch.zeros(nb, 2, KP, KP, dtype=pk.dtype,
                                 device=pk.device)
        for i, n in enumerate(("ra", "ri")):
            self.gates[:, i, :bw, :bw].copy_(pk.raw(p + n))
        self.cw = pk.f32(p + "conv").t().contiguous()
        self.cb = pk.f32(p + "conv.b")
        self.rb, self.ib = pk.f32(p + "ra.b"), pk.f32(p + "ri.b")
        lam = np.asarray(pk.w[p + "lam"], np.float64)
        self.nl = torch.from_numpy(
            (-s.C * np.logaddexp(lam, 0.0)).astype(np.float32)).to(pk.device)
        self.args = hy.RglruArgs().put(
            cw=self.cw, cb=self.cb, gates=self.gates, rb=self.rb, ib=self.ib,
            nl=self.nl, oy=0, ox=C, C=C, nb=nb, bw=bw, KP=KP, taps=s.conv,
            ldo=self.ldo)

    def new_cache(self, eng):
        n, s = eng.cache.num_slots, self.spec
        kw = dict(dtype=torch.float32, device=eng.device)
        return (torch.zeros(n, s.width, **kw),
                torch.zeros(n, s.conv, s.width, **kw))

    def sizes(self, eng, rows):
        C = self.spec.width
        return dict(o=rows * self.ldo, decay=rows * C, local=rows * C)

    def run(self, eng, b, cache, layer):
        nd = b.nd
        a = self.args.put(
            P=eng.P, S=cache[0], ring=cache[1], A=eng.decay, h=eng.local,
            out=eng.o, slot=b.slot, pos=b.pos, seg_row0=b.seg_row0[nd:],
            seg_len=b.seg_len[nd:], seg_slot=b.seg_slot[nd:],
            seg_pos0=b.seg_pos0[nd:], chunk_row0=b.chunk_row0,
            chunk_len=b.chunk_len, chunk_seg=b.chunk_seg, ldp=layer.ldp,
            rows=max(nd, 1), nchunk=b.nchunk)
        if nd:
            hy.rglru_step(eng.f32, a)
        if b.nseg:
            hy.rglru_run(eng.f32, a)


class Lightning(SandwichMixer):
    kind = "lightning"
    IN = ("q", "k", "v", "g")

    def __init__(self, eng, spec, pk: Packer, p: str):
        self.spec = s = spec
        H, d, vd = s.heads, s.dim, s.vdim
        if d > 8192:
            raise ValueError(f"lightning: dim {d} exceeds the built kernels")
        self.og = 2 * H * d + H * vd
        self.ldo = pad_to(H * vd, 64)
        self.wo = pk.rows([p + "o"], H * vd)
        self.norm = pk.f32(p + "norm")
        self.dpow = torch.from_numpy(
            (np.asarray(s.decay, np.float64)[:, None] **
             np.arange(hy.CHUNK + 1)).astype(np.float32)).to(pk.device)
        self.args = hy.LightningArgs().put(
            dpow=self.dpow, oq=0, ok=H * d, ov=2 * H * d, H=H, d=d, vd=vd,
            nvt=-(-vd // 64))

    def new_cache(self, eng):
        s = self.spec
        return (torch.zeros(eng.cache.num_slots, s.heads, s.dim, s.vdim,
                            dtype=torch.float32, device=eng.device),)

    def sizes(self, eng, rows):
        s = self.spec
        return dict(o=rows * self.ldo, raw=rows * s.heads * s.vdim,
                    U=eng.max_chunks(rows) * s.heads * s.dim * s.vdim)

    def run(self, eng, b, cache, layer):
        nd = b.nd
        a = self.args.put(
            P=eng.P, S=cache[0], o=eng.raw, U=eng.U, slot=b.slot, pos=b.pos,
            seg_len=b.seg_len[nd:], seg_slot=b.seg_slot[nd:],
            seg_pos0=b.seg_pos0[nd:], seg_chunk0=b.seg_chunk0,
            chunk_row0=b.chunk_row0, chunk_len=b.chunk_len, ldp=layer.ldp,
            rows=max(nd, 1), nseg=b.nseg, nchunk=b.nchunk)
        if nd:
            hy.lightning_step(a)
        if b.nseg:
            hy.lightning_run(a)

    def out(self, eng, b, layer):
        """All heads normed together, gated, projected."""
        eng.normed_linear(self.wo, eng.o, eng.y, b.T, eng.raw,
                          self.spec.heads * self.spec.vdim, self.norm,
                          gate=eng.P[self.og:], ldg=layer.ldp)


class InputConv:
    """A sublayer's input plus its causal convolution over time, channel by
    channel; a ring per sequence keeps the inputs that later steps need."""

    def __init__(self, pk: Packer, name: str):
        self.w = pk.f32(name).t().contiguous()         # [taps, width]

    def new_ring(self, eng):
        return torch.zeros(eng.cache.num_slots, *self.w.shape,
                           dtype=torch.float32, device=eng.device)


class DenseFF:
    """W_down act(W_up h); the hidden size is zero-padded to 64."""
    experts = None

    def __init__(self, eng, spec, pk: Packer, p: str):
        self.ff, self.ffp = spec.ff, pad_to(spec.ff, 64)
        up = pk.rows([p + "up"], eng.W)
        self.up = torch.zeros(self.ffp, up.shape[1], dtype=pk.dtype,
                              device=pk.device)
        self.up[:spec.ff].copy_(up)
        self.down = pk.rows([p + "down"], spec.ff)
        self.coef = pk.f32(p + "act") if spec.act == "polynorm" else None
        self.bias = self.down_bias = None
        if spec.act == "gelu":
            self.bias = torch.zeros(self.ffp, device=pk.device)
            self.bias[:spec.ff].copy_(pk.raw(p + "up.b"))
            self.down_bias = pk.f32(p + "down.b")
        self.act_floats = self.ffp
        self.p_floats = self.ffp if self.coef is not None else 0

    def after_up(self, eng, b, across):
        """eng.y from the up products in eng.P, a polynomial activation of
        the whole row between the two matrices."""
        eng.poly_linear(self.down, eng.P, self.ff, self.coef, eng.act,
                        eng.y, b.T)


class RoutedFF:
    """Routed experts of a block that does not route in its mixer."""

    def __init__(self, eng, spec, pk: Packer, p: str):
        self.experts = RoutedExperts(eng, spec, pk, p)
        self.up = pk.rows([p + "router"], eng.W)
        self.act_floats = self.experts.K1 * self.experts.ffm
        self.p_floats = spec.experts

    def after_up(self, eng, b, across):
        self.experts.apart(eng, b.T, b.nseg == 0, across)


FEED_FORWARDS = {"dense": DenseFF, "moe": RoutedFF}
MIXERS = {c.kind: c for c in (LatentAttention, MLSTM, GroupedAttention,
                              MinGRU, MixerPair, SSD, RGLRU, Lightning)}
