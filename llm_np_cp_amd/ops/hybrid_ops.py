"""ctypes bindings of the mixed-batch kernels: one library per mechanism
(csrc/linear.hip, latent_attn.hip, gqa_attn.hip, mlstm.hip, rglru.hip,
lightning.hip, moe.hip), each loaded when first used.

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
 EPI_ROTARY) = range(7)
ROW_NORM, ROW_CAT, ROW_PLAIN, ROW_CONV, ROW_POLY = range(5)
PAGE = 64           # tokens of a cache page (latent_attn.hip, gqa_attn.hip)
CHUNK = 64          # tokens of a chunk (linear, mlstm, rglru, lightning)
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
    (_p, "P qnorm knorm temp slot pos table K V q part ml o seg_row0 seg_len "
         "seg_slot seg_pos0 tile_seg tile_rr0"),
    (_i, "ldp oq ok ov og H G d vd DP VP ldo ldt rows rbase NS"),
    (_f, "eps scale"))
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
ConvRows = _struct(
    "ConvRows", (RowStage, "s"),
    (_p, "out seg_row0 seg_len seg_slot seg_pos0 chunk_row0 chunk_len "
         "chunk_seg"), (_i, "nd nseg nchunk"))
LinRowArgs = _struct(
    "LinRowArgs", (_p, "Wt"), (RowStage, "s"),
    (_p, "rows hin hout bias act y"), (_i, "N stage epi"), (_f, "cap"))
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
        "launch_norm_rows": [_i, _p, _p, _p, _i, _p],
        "launch_cat_rows": [_i, _p, _p, _p, _i, _i, _i, _p],
        "launch_lin_row": [_i, _p, _p],
        "launch_gemm_rows":
            [_i] + [_p] * 5 + [_i] * 8 + [_f, _i, _l, _l, _l, _i, _i, _p,
                                          _p],
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
        "launch_gqa_merge": [_i, _p, _p]},
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
            hin=None, res=None, gb=None, conv=None, act=None, **kw):
    """y[n] = Wt[n] . stage(x) [+ bias] for one row; stage is the norm of x
    with g or its convolution (see _stage; `res` is its y), the
    concatenation [x | x0], the polynomial activation of x with
    coefficients act, or the finished row hin.  hout receives the staged
    row (norm and convolution)."""
    N, Kp = Wt.shape
    stage = (ROW_NORM if g is not None else ROW_CAT if x0 is not None
             else ROW_CONV if conv is not None
             else ROW_POLY if act is not None else ROW_PLAIN)
    assert Kp % 64 == 0 and y.numel() >= N
    assert stage != ROW_PLAIN or hin.numel() >= Kp and hin.dtype == Wt.dtype
    assert stage != ROW_CAT or Kp >= 2 * W
    assert y.dtype == (Wt.dtype if epi == EPI_RELU2 else torch.float32)
    a = LinRowArgs().put(
        Wt=Wt, rows=_ptr(rows), hin=_ptr(hin), hout=_ptr(hout),
        bias=_ptr(bias), act=_ptr(act), y=y, N=N, stage=stage, epi=epi, cap=cap)
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
              bias=None, gz: int = 1, gc: int = 0, rotary=None):
    """Y[M, N] = X[M, K] Wt[N, K]^T with one of the EPI_* epilogues, for
    each of Z heads (element offsets xz/wz/yz).  Gates are at row*ldg +
    z*gz + column*gc.  EPI_ROTARY: the columns from rotary.split on go,
    rotated, to rotary.y."""
    N = N or Wt.shape[0]
    K = K or Wt.shape[-1]
    assert X.numel() >= (M - 1) * ldx + (Z - 1) * xz + K
    cols = rotary.split if epi == EPI_ROTARY else N
    assert Y.numel() >= (M - 1) * ldy + (Z - 1) * yz + cols
    assert Wt.numel() >= (Z - 1) * wz + N * K
    _go("launch_gemm_rows", _f32(Wt), _ptr(X), _ptr(Wt), _ptr(Y), _ptr(gate),
        _ptr(bias), M, N, K, ldx, K, ldy, ldg, epi, mult, Z, xz, wz, yz, gz, gc,
        ctypes.byref(rotary) if rotary is not None else 0)


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


def gqa_merge(f32, a):
    _go("launch_gqa_merge", f32, ctypes.byref(a))


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
