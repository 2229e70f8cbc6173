"""ctypes bindings of the mixed-batch kernels: one library per mechanism
(csrc/linear.hip, latent_attn.hip, gqa_attn.hip, mlstm.hip, mingru.hip,
ssd.hip, rglru.hip, lightning.hip, moe.hip), each loaded when first used.

Tensors are memory containers; launches land on the current torch stream.
Argument blocks are C structs filled from tensors and ints; shapes are
checked here and again in the launchers before anything runs.
"""

from __future__ import annotations

import ctypes
import os

import torch

_PKG = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
_FNS = {}

(EPI_F32, EPI_RESADD, EPI_SOFTCAP, EPI_T, EPI_TGATE, EPI_RELU2,
 EPI_ROTARY, EPI_GELU) = range(8)
(ROW_NORM, ROW_CAT, ROW_PLAIN, ROW_CONV, ROW_POLY, ROW_HYPER,
 ROW_GROUPS) = range(7)
PAGE = 64           # tokens of a cache page (latent_attn.hip, gqa_attn.hip)
CHUNK = 64          # tokens of a chunk (linear and the recurrences)
MAX_STREAMS = 8     # residual streams (linear.hip)
MAX_GROUPS = 1024   # parts of a norm (linear.hip)
MAX_SPLITS = 256
TILE = 64           # (token, head) pairs of an attention block over runs
RANKS = (64, 128, 256, 384, 512)      # padded latent sizes that are built
# padded (key, value) sizes of a grouped-query head that are built
HEAD_SIZES = ((64, 64), (64, 128), (128, 64), (128, 128), (256, 256))

_p, _i, _l, _f = (ctypes.c_void_p, ctypes.c_int, ctypes.c_long,
                  ctypes.c_float)


class _Args(ctypes.Structure):
    """Fill from tensors / numbers; unknown names are an error."""

    def put(self, **kw):
        names = self._names
        for k, v in kw.items():
            if k not in names:
                raise AttributeError(k)
            if isinstance(v, torch.Tensor):
                v = v.data_ptr()
            setattr(self, k, v)
        return self


def _struct(name, *fields):
    fl = [(n, t) for t, names in fields for n in names.split()]
    return type(name, (_Args,), {"_fields_": fl,
                                 "_names": {n for n, _ in fl}})


LatentArgs = _struct(
    "LatentArgs",
    (_p, "P Q cq qnorm sink Wuk Wuv cnorm cosT sinT slot pos table cache qn qa part ml olat "
         "o seg_row0 seg_len seg_slot seg_pos0 tile_seg tile_rr0 ridx rwt"),
    (_i, "ldp oq odkv og orouter H d dp rot rdims RT rank RP vd ldo ldt rows "
         "rbase NS E rtop rextra ldq qh oqr qrh qrank QRp pairs win gz gc "
         "written"),
    (_f, "eps scale"))
MlstmArgs = _struct(
    "MlstmArgs",
    (_p, "P ib fb norm S n m o out slot pos seg_row0 seg_len seg_slot "
         "seg_pos0 seg_chunk0 chunk_row0 chunk_len gF gi gm cm0 U un ridx "
         "rwt"),
    (_i, "ldp oq ok ov og oi of orouter H d vd nvt ldo rows nseg nchunk E "
         "rtop rextra"),
    (_f, "cap eps"))
GqaArgs = _struct(
    "GqaArgs",
    (_p, "P qnorm knorm temp bias sink slot pos table K V q part ml o seg_row0 "
         "seg_len seg_slot seg_pos0 tile_seg tile_rr0"),
    (_i, "ldp oq ok ov og H G d vd DP VP ldo ldt rows rbase NS chunk nbias"),
    (_f, "eps scale"))
MingruArgs = _struct(
    "MingruArgs",
    (_p, "P S A h out slot pos seg_row0 seg_len seg_slot seg_pos0 chunk_row0 "
         "chunk_len chunk_seg"),
    (_i, "ldp oz ox og C ldo rows nchunk"))
SsdArgs = _struct(
    "SsdArgs",
    (_p, "P cw cb dtb rate D S ring u dt L U o slot pos seg_row0 seg_len "
         "seg_slot seg_pos0 seg_chunk0 chunk_row0 chunk_len chunk_seg"),
    (_i, "ldp oz ox odt H G N vd C taps nvt rows nseg nchunk"))
RglruArgs = _struct(
    "RglruArgs",
    (_p, "P cw cb gates rb ib nl S ring A h out slot pos seg_row0 seg_len "
         "seg_slot seg_pos0 chunk_row0 chunk_len chunk_seg"),
    (_i, "ldp oy ox C nb bw KP taps ldo rows nchunk"))
LightningArgs = _struct(
    "LightningArgs",
    (_p, "P dpow S o U slot pos seg_len seg_slot seg_pos0 seg_chunk0 "
         "chunk_row0 chunk_len"),
    (_i, "ldp oq ok ov H d vd nvt rows nseg nchunk"))
RowStage = _struct(
    "RowStage", (_p, "x y gb xadd g gate xout cw ring slot pos"),
    (_i, "W Kp ldg taps"), (_f, "eps"))
HyperStage = _struct(
    "HyperStage", (_p, "x y y2 gb gb2 mix feed in_ g xout"), (_i, "W Kp S"),
    (_f, "eps"))
PairEmbed = _struct(
    "PairEmbed", (_p, "table pairs ids slot pos last x seg_row0 seg_len "
                      "seg_slot"), (_l, "mul_before mul_cur"),
    (_i, "W S M nd nseg buckets"))
ConvRows = _struct(
    "ConvRows", (RowStage, "s"),
    (_p, "out seg_row0 seg_len seg_slot seg_pos0 chunk_row0 chunk_len "
         "chunk_seg"), (_i, "nd nseg nchunk"))
LinRowArgs = _struct(
    "LinRowArgs", (_p, "Wt"), (RowStage, "s"),
    (_p, "rows hin hout bias act y"), (_i, "N stage epi"), (_f, "cap"),
    (_i, "groups Z K2"), (_l, "xz wz yz"), (HyperStage, "h"))
Rotary = _struct(
    "Rotary", (_p, "pos cosT sinT y"), (_i, "split RT dims ld hs"))
MoeArgs = _struct(
    "MoeArgs", (_p, "h gu down idx wt act"),
    (_i, "ldh ldact W E K1 ff ffs glu win"), (_f, "lim lims"))
RouteArgs = _struct(
    "RouteArgs", (_p, "z idx wt"), (_i, "ldz lde rows E top extra scores"))
MoeSort = _struct(
    "MoeSort", (_p, "perm tile_e tile_row0 tile_n"),
    (_i, "pairs groups bm maxtiles"))

_SIGS = {
    "linear": {
        "launch_embed_rows": [_i, _p, _p, _p, _p, _i, _i, _f, _p],
        "launch_embed_pairs": [_i, _p, _p],
        "launch_hyper_rows": [_i, _p, _p, _p, _i, _p],
        "launch_group_rows": [_i, _p, _i, _p, _i, _p],
        "launch_norm_rows": [_i, _p, _p, _p, _i, _p],
        "launch_cat_rows": [_i, _p, _p, _p, _i, _i, _i, _p],
        "launch_lin_row": [_i, _p, _p],
        "launch_gemm_rows":
            [_i] + [_p] * 5 + [_i] * 8 + [_f, _i, _l, _l, _l, _i, _i, _p,
                                          _i, _p],
        "launch_conv_rows": [_i, _p, _p],
        "launch_poly_rows": [_i, _p, _i, _p, _p, _i, _i, _i, _f, _p]},
    "latent": {
        "launch_latent_prep": [_i, _p, _p],
        "launch_latent_mid": [_i, _p, _p],
        "launch_latent_dec_prep": [_i, _p, _p],
        "launch_latent_attn": [_i, _p, _i, _i, _p],
        "launch_latent_merge": [_i, _p, _p],
        "launch_latent_dec_fin": [_i, _p, _p, _i, _p]},
    "gqa": {
        "launch_gqa_prep": [_i, _p, _p],
        "launch_gqa_token": [_i, _p, _p],
        "launch_gqa_run": [_i, _p, _i, _p],
        "launch_gqa_merge": [_i, _p, _p, _p]},
    "mingru": {
        "launch_mingru_step": [_i, _p, _p],
        "launch_mingru_run": [_i, _p, _p]},
    "ssd": {
        "launch_ssd_step": [_p, _p],
        "launch_ssd_run": [_p, _p]},
    "mlstm": {
        "launch_mlstm_step": [_p, _p],
        "launch_mlstm_chunks": [_p, _p],
        "launch_mlstm_post": [_i, _p, _p],
        "launch_mlstm_dec_fin": [_i, _p, _p, _i, _p]},
    "rglru": {
        "launch_rglru_step": [_i, _p, _p],
        "launch_rglru_run": [_i, _p, _p]},
    "lightning": {
        "launch_lightning_step": [_p, _p],
        "launch_lightning_run": [_p, _p]},
    "moe": {
        "launch_block_out": [_i, _p, _p, _i, _p, _i, _p, _i, _i, _f, _i, _p],
        "launch_moe_gu_few": [_i, _p, _p, _p],
        "launch_moe_route": [_p, _p, _p],
        "launch_moe_rows": [_i, _p, _p, _p, _p, _i, _f, _i, _p]},
}
_LIB_OF = {fn: name for name, sigs in _SIGS.items() for fn in sigs}


def _fn(launcher):
    if launcher not in _FNS:
        name = _LIB_OF[launcher]
        path = os.path.join(_PKG, f"_lib{name}.so")
        if not os.path.exists(path):
            raise RuntimeError(
                f"HIP kernel library not built: {path} missing. "
                f"Run `python csrc/build.py` (or __graft_entry__.build()).")
        lib = ctypes.CDLL(path)
        for fn, argtypes in _SIGS[name].items():
            f = getattr(lib, fn)
            f.argtypes = argtypes
            f.restype = ctypes.c_int
            _FNS[fn] = f
    return _FNS[launcher]


def _go(name, *args):
    err = _fn(name)(*args, torch.cuda.current_stream().cuda_stream)
    if err != 0:
        raise RuntimeError(f"{name} failed: hipError_t={err}")


def _ptr(t):
    return 0 if t is None else t.data_ptr()


def _f32(t: torch.Tensor) -> int:
    assert t.dtype in (torch.float32, torch.bfloat16), t.dtype
    return 1 if t.dtype == torch.float32 else 0


def embed_rows(table, ids, x, x0, M: int, scale: float):
    """x[r] = table[ids[r]] * scale in fp32 (and a copy in x0)."""
    W = table.shape[1]
    assert x.numel() >= M * W and (x0 is None or x0.numel() >= M * W)
    _go("launch_embed_rows", _f32(table), _ptr(table), _ptr(ids), _ptr(x),
        _ptr(x0), M, W, scale)


def embed_pairs(table, pairs, last, b, x, W: int, S: int, spec):
    """x[r] (S streams) = table[id] + the row of pairs for the token before
    it and this one; `last` [slots] holds the token before each sequence's
    next one and moves on."""
    assert table.shape[1] == pairs.shape[1] == W
    assert pairs.shape[0] == spec.buckets + 1 and x.numel() >= b.T * S * W
    a = PairEmbed().put(
        table=table, pairs=pairs, ids=b.ids, slot=b.slot, pos=b.pos,
        last=last, x=x, seg_row0=b.seg_row0[b.nd:], seg_len=b.seg_len[b.nd:],
        seg_slot=b.seg_slot[b.nd:], mul_before=spec.mul_prev,
        mul_cur=spec.mul_cur, W=W, S=S, M=b.T, nd=b.nd, nseg=b.nseg,
        buckets=spec.buckets)
    _go("launch_embed_pairs", _f32(table), ctypes.byref(a))


def _hyper(x, W: int, Kp: int, eps: float, S: int, read=None, g=None,
           y=None, y2=None, gb=None, gb2=None, mix=None, feed=None,
           xout=None):
    """Staging of rows of S streams: with y (and y2: half the sum of both,
    normed with weights gb, gb2) the streams turn by mix and feed; then
    u = their sum weighted by read, u/rms(u) times the number g."""
    assert mix is None or mix.shape == (S, S)
    return HyperStage().put(
        x=_ptr(x), y=_ptr(y), y2=_ptr(y2), gb=_ptr(gb), gb2=_ptr(gb2),
        mix=_ptr(mix), feed=_ptr(feed), in_=_ptr(read), g=_ptr(g),
        xout=_ptr(xout), W=W, Kp=Kp, S=S, eps=eps)


def hyper_rows(x, out, M: int, W: int, Kp: int, eps: float, S: int,
               rows=None, **kw):
    """Staged rows (see _hyper) [M, Kp], zero beyond W; takes read, g, y,
    y2, gb, gb2, mix, feed, xout (x itself is allowed).  Without read only
    xout is written."""
    assert out is None or out.numel() >= M * Kp
    s = _hyper(x, W, Kp, eps, S, **kw)
    _go("launch_hyper_rows", 0 if out is None else _f32(out),
        ctypes.byref(s), _ptr(rows), _ptr(out), M)


def group_rows(x, g, out, M: int, W: int, Kp: int, eps: float, groups: int):
    """Rows of x normed in equal parts, times g -> out [M, Kp]."""
    assert x.numel() >= M * W and out.numel() >= M * Kp
    s = RowStage().put(x=x, g=g, W=W, Kp=Kp, eps=eps)
    _go("launch_group_rows", _f32(out), ctypes.byref(s), groups, _ptr(out),
        M)


def _stage(x, W: int, Kp: int, eps: float, g=None, y=None, gb=None,
           xadd=None, gate=None, ldg: int = 0, xout=None, conv=None):
    """Staging of residual rows: v = x [+ y/rms(y) gb] [+ xadd], then
    v/rms(v) g [sigmoid(gate)]; xout receives v.  conv = (kernel [taps, W],
    ring [slots, taps, W], slots, positions): v + its convolution over time
    instead of the norm."""
    assert (y is None) == (gb is None) and (g is None or Kp >= W)
    s = RowStage().put(x=_ptr(x), y=_ptr(y), gb=_ptr(gb), xadd=_ptr(xadd),
                       g=_ptr(g), gate=_ptr(gate), xout=_ptr(xout), W=W,
                       Kp=Kp, ldg=ldg, eps=eps)
    if conv is not None:
        cw, ring, slot, pos = conv
        assert cw.shape[1] == W and ring.shape[1:] == cw.shape
        s.put(cw=cw, ring=ring, slot=slot, pos=pos, taps=cw.shape[0])
    return s


def norm_rows(x, g, out, M: int, W: int, Kp: int, eps: float, rows=None,
              x0=None, **kw):
    """Staged rows (see _stage) [M, Kp], zero beyond W, from the rows of x
    (or those that `rows` picks); takes y, gb, xadd, gate, ldg, xout (x
    itself is allowed).  Without g: [x | x0], or, without x0 either, only
    xout is written."""
    assert out is None or out.numel() >= M * Kp
    if x0 is not None:
        assert g is None and rows is None and not kw and Kp >= 2 * W
        _go("launch_cat_rows", _f32(out), _ptr(x), _ptr(x0), _ptr(out), M, W,
            Kp)
        return
    s = _stage(x, W, Kp, eps, g, **kw)
    _go("launch_norm_rows", 0 if out is None else _f32(out), ctypes.byref(s),
        _ptr(rows), _ptr(out), M)


def lin_row(Wt, x, y, W: int, eps: float, g=None, x0=None, rows=None,
            hout=None, cap: float = 0.0, bias=None, epi: int = EPI_F32,
            hin=None, res=None, gb=None, conv=None, act=None, hyper=None,
            groups: int = 0, second=None, **kw):
    """y[n] = Wt[n] . stage(x) [+ bias] for one row; stage is the norm of x
    with g or its convolution (see _stage; `res` is its y), the
    concatenation [x | x0], the polynomial activation of x with
    coefficients act, the streams x turned and read as `hyper` says
    (arguments of _hyper), the norm with g in `groups` parts, or the
    finished row hin.  hout receives the staged row (norm, convolution,
    streams).  second = (K, element offsets of row, weights and y): another
    product with a finished row in the same launch."""
    N, Kp = Wt.shape
    stage = (ROW_HYPER if hyper is not None else ROW_GROUPS if groups > 1
             else ROW_NORM if g is not None else ROW_CAT if x0 is not None
             else ROW_CONV if conv is not None
             else ROW_POLY if act is not None else ROW_PLAIN)
    assert Kp % 64 == 0 and y.numel() >= N
    assert stage != ROW_PLAIN or hin.numel() >= Kp and hin.dtype == Wt.dtype
    assert stage != ROW_CAT or Kp >= 2 * W
    assert y.dtype == (Wt.dtype if epi in (EPI_RELU2, EPI_GELU)
                       else torch.float32)
    a = LinRowArgs().put(
        Wt=Wt, rows=_ptr(rows), hin=_ptr(hin), hout=_ptr(hout),
        bias=_ptr(bias), act=_ptr(act), y=y, N=N, stage=stage, epi=epi,
        cap=cap, groups=groups, Z=1)
    if second is not None:
        K2, xz, wz, yz = second
        assert stage == ROW_PLAIN and hin.numel() >= xz + K2
        assert y.numel() >= yz + N
        a.put(Z=2, K2=K2, xz=xz, wz=wz, yz=yz)
    if hyper is not None:
        a.h = _hyper(x, W, Kp, eps, **hyper)
    if stage == ROW_CAT:
        kw["xadd"] = x0
    a.s = _stage(x, W, Kp, eps, g, y=res, gb=gb, conv=conv, **kw)
    _go("launch_lin_row", _f32(Wt), ctypes.byref(a))


def conv_rows(x, out, b, W: int, Kp: int, eps: float, conv, **kw):
    """out[r] = v + conv(v) for the rows of batch b (see _stage; takes y,
    gb, xout)."""
    assert out.numel() >= b.T * Kp and Kp % 64 == 0
    nd = b.nd
    a = ConvRows().put(
        out=out, seg_row0=b.seg_row0[nd:], seg_len=b.seg_len[nd:],
        seg_slot=b.seg_slot[nd:], seg_pos0=b.seg_pos0[nd:],
        chunk_row0=b.chunk_row0, chunk_len=b.chunk_len, chunk_seg=b.chunk_seg,
        nd=nd, nseg=b.nseg, nchunk=b.nchunk)
    a.s = _stage(x, W, Kp, eps, conv=conv, **kw)
    _go("launch_conv_rows", _f32(out), ctypes.byref(a))


def poly_rows(z, ldz: int, act, out, M: int, W: int, eps: float):
    """out[M, W padded to 64] = a N(z) + b N(z^2) + c N(z^3) + e."""
    Kp = -(-W // 64) * 64
    assert z.numel() >= (M - 1) * ldz + W and out.numel() >= M * Kp
    _go("launch_poly_rows", _f32(out), _ptr(z), ldz, _ptr(act), _ptr(out), M,
        W, Kp, eps)


def gemm_rows(X, Wt, Y, M: int, ldx: int, ldy: int, epi: int,
              mult: float = 0.0, N: int = 0, K: int = 0, Z: int = 1,
              xz: int = 0, wz: int = 0, yz: int = 0, gate=None, ldg: int = 0,
              bias=None, gz: int = 1, gc: int = 0, rotary=None,
              K2: int = 0):
    """Y[M, N] = X[M, K] Wt[N, K]^T with one of the EPI_* epilogues, for
    each of Z heads (element offsets xz/wz/yz; K2: the K of those after the
    first, where it differs).  Gates are at row*ldg +
    z*gz + column*gc.  EPI_ROTARY: the columns from rotary.split on go,
    rotated, to rotary.y."""
    N = N or Wt.shape[0]
    K = K or Wt.shape[-1]
    KZ = K2 or K
    assert X.numel() >= (M - 1) * ldx + max(K, (Z - 1) * xz + KZ)
    cols = rotary.split if epi == EPI_ROTARY else N
    assert Y.numel() >= (M - 1) * ldy + (Z - 1) * yz + cols
    assert Wt.numel() >= max(N * K, (Z - 1) * wz + N * KZ)
    _go("launch_gemm_rows", _f32(Wt), _ptr(X), _ptr(Wt), _ptr(Y), _ptr(gate),
        _ptr(bias), M, N, K, ldx, K, ldy, ldg, epi, mult, Z, xz, wz, yz, gz, gc,
        ctypes.byref(rotary) if rotary is not None else 0, KZ)


def latent_prep(f32, a):
    _go("launch_latent_prep", f32, ctypes.byref(a))


def latent_mid(f32, a):
    _go("launch_latent_mid", f32, ctypes.byref(a))


def latent_dec_prep(f32, a):
    _go("launch_latent_dec_prep", f32, ctypes.byref(a))


def latent_attn(f32, a, share: int, tiles: int):
    """tiles of 16 (share: single tokens) or 64 (token, head) pairs."""
    _go("launch_latent_attn", f32, ctypes.byref(a), share, tiles)


def latent_merge(f32, a):
    _go("launch_latent_merge", f32, ctypes.byref(a))


def latent_dec_fin(f32, a, m, pairs: int):
    _go("launch_latent_dec_fin", f32, ctypes.byref(a), ctypes.byref(m), pairs)


def gqa_prep(f32, a):
    _go("launch_gqa_prep", f32, ctypes.byref(a))


def gqa_token(f32, a):
    _go("launch_gqa_token", f32, ctypes.byref(a))


def gqa_run(f32, a, tiles: int):
    """tiles of TILE (token, head of the group) pairs."""
    _go("launch_gqa_run", f32, ctypes.byref(a), tiles)


def gqa_merge(f32, a, beside=None):
    """beside: single tokens of a gated recurrence (MingruArgs) that take
    their step in the same launch."""
    _go("launch_gqa_merge", f32, ctypes.byref(a),
        0 if beside is None else ctypes.byref(beside))


def mingru_step(f32, a):
    _go("launch_mingru_step", f32, ctypes.byref(a))


def mingru_run(f32, a):
    _go("launch_mingru_run", f32, ctypes.byref(a))


def ssd_step(a):
    _go("launch_ssd_step", ctypes.byref(a))


def ssd_run(a):
    _go("launch_ssd_run", ctypes.byref(a))


def rglru_step(f32, a):
    _go("launch_rglru_step", f32, ctypes.byref(a))


def rglru_run(f32, a):
    _go("launch_rglru_run", f32, ctypes.byref(a))


def lightning_step(a):
    _go("launch_lightning_step", ctypes.byref(a))


def lightning_run(a):
    _go("launch_lightning_run", ctypes.byref(a))


def mlstm_step(a):
    _go("launch_mlstm_step", ctypes.byref(a))


def mlstm_chunks(a):
    _go("launch_mlstm_chunks", ctypes.byref(a))


def mlstm_post(f32, a):
    _go("launch_mlstm_post", f32, ctypes.byref(a))


def mlstm_dec_fin(f32, a, m, pairs: int):
    _go("launch_mlstm_dec_fin", f32, ctypes.byref(a), ctypes.byref(m), pairs)


def block_out(f32, Wo, o, ldo: int, m, K1: int, x, rows: int, W: int,
              mult: float, set: bool = False):
    """x[r] += mult (Wo o_r + the experts' outputs), or with `set` x[r] =
    that; without Wo where ldo is 0."""
    _go("launch_block_out", f32, _ptr(Wo), _ptr(o), ldo, ctypes.byref(m), K1,
        _ptr(x), rows, W, mult, int(set))


def moe_gu_few(f32, m, route):
    """Routing and the experts' gate/up halves, one block row per pair."""
    _go("launch_moe_gu_few", f32, ctypes.byref(m), ctypes.byref(route))


def moe_route(m, route):
    _go("launch_moe_route", ctypes.byref(m), ctypes.byref(route))


def moe_rows(f32, m, s, y, x, rows: int, mult: float, set: bool = False):
    _go("launch_moe_rows", f32, ctypes.byref(m), ctypes.byref(s), _ptr(y),
        _ptr(x), rows, mult, int(set))
