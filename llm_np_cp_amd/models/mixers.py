"""Device side of the layer-list mechanisms: weights in kernel layout, the
cache or state of each layer run, and the kernel sequence for a batch.

Every mechanism has two sequences over the same cache and state:

    few()   up to 16 rows, one token each (decode): fused small launches;
            with `fuse` the experts' gate/up halves ride along
    many()  any mix of single tokens and runs of tokens: MFMA GEMMs, run
            kernels over the runs, single-token kernels over the rest

A batch lists its single-token rows first.  Both leave the mixer's output
(before the output projection) in eng.o and the expert choice in
eng.ridx / eng.rwt.
"""

from __future__ import annotations

import torch

from ..ops import hybrid_ops as hy


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
    """Clamped-GLU experts and their shared one (see csrc/moe.h for the
    weight layout); routing logits are columns of the block's input
    projection, so the router costs no launch of its own."""

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
            K1=self.K1, ff=ff, ffs=ffs, lim=spec.expert.limit,
            lims=sh.limit if sh else 0.0)

    def bind(self, eng):
        return self.args.put(h=eng.h, idx=eng.ridx, wt=eng.rwt, act=eng.act)

    def many(self, eng, T: int):
        avg = T * self.top / self.spec.experts
        bm = 128 if avg >= 160 else 64 if avg >= 24 else 32
        pairs, groups = T * self.K1, self.spec.experts + self.extra
        s = hy.MoeSort().put(
            perm=eng.perm, tile_e=eng.tile_e, tile_row0=eng.tile_row0,
            tile_n=eng.tile_n, pairs=pairs, groups=groups, bm=bm,
            maxtiles=pairs // bm + groups)
        assert s.maxtiles <= eng.tile_e.numel()
        hy.moe_rows(eng.f32, self.bind(eng), s, eng.ypair, eng.x, T,
                    eng.cfg.residual_mult)


class LatentAttention:
    kind = "latent_attention"
    IN = ("q", "dkv", "g")           # rows of the input projection

    def __init__(self, eng, spec, pk: Packer, p: str):
        self.spec = s = spec
        fit = [r for r in hy.RANKS if r >= s.kv_rank]
        if not fit or s.rot_dim > 128:
            raise ValueError(
                f"latent attention: kv_rank {s.kv_rank} / rot_dim "
                f"{s.rot_dim} exceed the built kernels "
                f"({hy.RANKS[-1]} / 128)")
        self.RP, self.RT = fit[0], pad_to(s.rot_dim, 32)
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
        nq = H * (d + s.rot_dim)
        self.args = hy.LatentArgs().put(
            Wuk=self.wuk, Wuv=self.wuv, cnorm=self.cnorm, cosT=self.cosT,
            sinT=self.sinT, oq=0, odkv=nq, og=nq + s.kv_rank + s.rot_dim,
            H=H, d=d, dp=self.dp, rot=s.rot_dim, rdims=s.rot_dims,
            RT=self.RT, rank=s.kv_rank, RP=RP, vd=vd, ldo=self.ldo,
            eps=eng.cfg.norm_eps, scale=s.scale)

    def new_cache(self, eng):
        return torch.zeros(eng.cache.num_pages, hy.PAGE, self.CS,
                           dtype=eng.T, device=eng.device)

    def sizes(self, rows, splits):
        """Scratch elements for `rows` rows (fp32 partials for splits)."""
        H = self.spec.heads
        return dict(qn=rows * H * self.dp, qa=rows * H * self.CS,
                    olat=rows * H * self.RP, o=rows * self.ldo,
                    part=splits * H * self.RP, ml=splits * H * 2)

    def _bind(self, eng, b, cache, layer):
        x = layer.experts
        return self.args.put(
            P=eng.P, slot=b.slot, pos=b.pos, table=eng.table, cache=cache,
            qn=eng.qn, qa=eng.qa, part=eng.part, ml=eng.ml, olat=eng.olat,
            o=eng.o, seg_row0=b.seg_row0, seg_len=b.seg_len,
            seg_slot=b.seg_slot, seg_pos0=b.seg_pos0, tile_seg=0,
            tile_rr0=0, ridx=eng.ridx, rwt=eng.rwt, ldp=layer.ldp,
            orouter=layer.orouter, ldt=eng.table.shape[1], rows=b.T, rbase=0,
            NS=1, E=x.spec.experts if x else 0, rtop=x.top if x else 0,
            rextra=x.extra if x else 0)

    def _single(self, eng, a, n):
        """Split attention of the first n rows, partials left in part/ml."""
        a.put(rows=n, rbase=0, NS=eng.decode_splits(n))
        hy.latent_attn(eng.f32, a, 1, n * (-(-self.spec.heads // 16)))

    def few(self, eng, b, cache, layer, fuse):
        a = self._bind(eng, b, cache, layer)
        hy.latent_dec_prep(eng.f32, a)
        self._single(eng, a, b.T)
        x = layer.experts if fuse else None
        hy.latent_dec_fin(eng.f32, a, x.bind(eng) if x else hy.MoeArgs(),
                          b.T * x.K1 if x else 0)

    def many(self, eng, b, cache, layer):
        s, H, CS, RP = self.spec, self.spec.heads, self.CS, self.RP
        a = self._bind(eng, b, cache, layer)
        hy.latent_prep(eng.f32, a)
        hy.gemm_rows(eng.qn, self.wukT, eng.qa, b.T, H * self.dp, H * CS,
                     hy.EPI_T, N=RP, K=self.dp, Z=H, xz=self.dp,
                     wz=RP * self.dp, yz=CS)
        if b.nd:
            self._single(eng, a, b.nd)
            hy.latent_merge(eng.f32, a)
        if b.nd < b.T:
            seg, rr0, n, longest = b.tiles[H]
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
                     wz=s.vdim * RP, yz=s.vdim,
                     gate=eng.P[a.og:], ldg=layer.ldp)


class MLSTM:
    kind = "mlstm"
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

    def sizes(self, rows, splits):
        s, chunks = self.spec, rows // hy.CHUNK + splits
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


MIXERS = {c.kind: c for c in (LatentAttention, MLSTM)}
