"""ctypes bindings of the mixed-batch kernels (``_libhybrid.so``:
csrc/linear.hip, latent_attn.hip, mlstm.hip, moe.hip).

Tensors are memory containers; launches land on the current torch stream.
Argument blocks are C structs filled from tensors and ints; shapes are
checked here and again in the launchers before anything runs.
"""

from __future__ import annotations

import ctypes
import os

import torch

_LIB = None
_LIB_PATH = os.path.join(os.path.dirname(os.path.dirname(
    os.path.abspath(__file__))), "_libhybrid.so")

EPI_F32, EPI_RESADD, EPI_SOFTCAP, EPI_T, EPI_TGATE = range(5)
PAGE = 64           # tokens of a cache page (latent_attn.hip)
CHUNK = 64          # tokens of a recurrence chunk (mlstm.hip)
MAX_SPLITS = 256
RANKS = (64, 128, 256, 384, 512)      # padded latent sizes that are built

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
    (_p, "P Wuk Wuv cnorm cosT sinT slot pos table cache qn qa part ml olat "
         "o seg_row0 seg_len seg_slot seg_pos0 tile_seg tile_rr0 ridx rwt"),
    (_i, "ldp oq odkv og orouter H d dp rot rdims RT rank RP vd ldo ldt rows "
         "rbase NS E rtop rextra"),
    (_f, "eps scale"))
MlstmArgs = _struct(
    "MlstmArgs",
    (_p, "P ib fb norm S n m o out slot pos seg_row0 seg_len seg_slot "
         "seg_pos0 seg_chunk0 chunk_row0 chunk_len gF gi gm cm0 U un ridx "
         "rwt"),
    (_i, "ldp oq ok ov og oi of orouter H d vd nvt ldo rows nseg nchunk E "
         "rtop rextra"),
    (_f, "cap eps"))
MoeArgs = _struct(
    "MoeArgs", (_p, "h gu down idx wt act"),
    (_i, "ldh ldact W E K1 ff ffs"), (_f, "lim lims"))
MoeSort = _struct(
    "MoeSort", (_p, "perm tile_e tile_row0 tile_n"),
    (_i, "pairs groups bm maxtiles"))

_SIGS = {
    "launch_embed_rows": [_i, _p, _p, _p, _p, _i, _i, _f, _p],
    "launch_norm_rows": [_i, _p, _p, _p, _p, _p, _i, _i, _i, _f, _p],
    "launch_lin_row": [_i] + [_p] * 7 + [_i] * 3 + [_f, _f, _p],
    "launch_gemm_rows": [_i] + [_p] * 4 + [_i] * 8 + [_f, _i, _l, _l, _l, _p],
    "launch_latent_prep": [_i, _p, _p],
    "launch_latent_dec_prep": [_i, _p, _p],
    "launch_latent_attn": [_i, _p, _i, _i, _p],
    "launch_latent_merge": [_i, _p, _p],
    "launch_latent_dec_fin": [_i, _p, _p, _i, _p],
    "launch_mlstm_step": [_p, _p],
    "launch_mlstm_chunks": [_p, _p],
    "launch_mlstm_post": [_i, _p, _p],
    "launch_mlstm_dec_fin": [_i, _p, _p, _i, _p],
    "launch_block_out": [_i, _p, _p, _i, _p, _i, _p, _i, _i, _f, _p],
    "launch_moe_rows": [_i, _p, _p, _p, _p, _i, _f, _p],
}


def lib():
    global _LIB
    if _LIB is None:
        if not os.path.exists(_LIB_PATH):
            raise RuntimeError(
                f"HIP kernel library not built: {_LIB_PATH} missing. "
                f"Run `python csrc/build.py` (or __graft_entry__.build()).")
        _LIB = ctypes.CDLL(_LIB_PATH)
        for name, argtypes in _SIGS.items():
            fn = getattr(_LIB, name)
            fn.argtypes = argtypes
            fn.restype = ctypes.c_int
    return _LIB


def _go(name, *args):
    err = getattr(lib(), name)(*args, torch.cuda.current_stream().cuda_stream)
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


def norm_rows(x, g, out, M: int, W: int, Kp: int, eps: float, rows=None,
              x0=None):
    """out[r, :Kp] = rmsnorm(x[rows[r]]) * g, or [x | x0] when g is None;
    zero beyond the row."""
    assert out.numel() >= M * Kp and (g is not None or x0 is not None)
    assert Kp >= (W if g is not None else 2 * W)
    _go("launch_norm_rows", _f32(out), _ptr(x), _ptr(x0), _ptr(g),
        _ptr(rows), _ptr(out), M, W, Kp, eps)


def lin_row(Wt, x, y, W: int, eps: float, g=None, x0=None, rows=None,
            hout=None, cap: float = 0.0):
    """y[n] = Wt[n] . stage(x) for one row; stage = norm (g) or the
    concatenation [x | x0].  hout receives the staged row."""
    N, Kp = Wt.shape
    assert Kp % 64 == 0 and Kp >= (W if g is not None else 2 * W)
    assert y.numel() >= N and y.dtype == torch.float32
    _go("launch_lin_row", _f32(Wt), _ptr(Wt), _ptr(x), _ptr(x0), _ptr(g),
        _ptr(rows), _ptr(hout), _ptr(y), N, W, Kp, eps, cap)


def gemm_rows(X, Wt, Y, M: int, ldx: int, ldy: int, epi: int,
              mult: float = 0.0, N: int = 0, K: int = 0, Z: int = 1,
              xz: int = 0, wz: int = 0, yz: int = 0, gate=None, ldg: int = 0):
    """Y[M, N] = X[M, K] Wt[N, K]^T with one of the EPI_* epilogues, for
    each of Z heads (element offsets xz/wz/yz)."""
    N = N or Wt.shape[0]
    K = K or Wt.shape[-1]
    assert X.numel() >= (M - 1) * ldx + (Z - 1) * xz + K
    assert Y.numel() >= (M - 1) * ldy + (Z - 1) * yz + N
    assert Wt.numel() >= (Z - 1) * wz + N * K
    _go("launch_gemm_rows", _f32(Wt), _ptr(X), _ptr(Wt), _ptr(Y), _ptr(gate),
        M, N, K, ldx, K, ldy, ldg, epi, mult, Z, xz, wz, yz)


def latent_prep(f32, a):
    _go("launch_latent_prep", f32, ctypes.byref(a))


def latent_dec_prep(f32, a):
    _go("launch_latent_dec_prep", f32, ctypes.byref(a))


def latent_attn(f32, a, share: int, tiles: int):
    """tiles of 16 (share: single tokens) or 64 (token, head) pairs."""
    _go("launch_latent_attn", f32, ctypes.byref(a), share, tiles)


def latent_merge(f32, a):
    _go("launch_latent_merge", f32, ctypes.byref(a))


def latent_dec_fin(f32, a, m, pairs: int):
    _go("launch_latent_dec_fin", f32, ctypes.byref(a), ctypes.byref(m), pairs)


def mlstm_step(a):
    _go("launch_mlstm_step", ctypes.byref(a))


def mlstm_chunks(a):
    _go("launch_mlstm_chunks", ctypes.byref(a))


def mlstm_post(f32, a):
    _go("launch_mlstm_post", f32, ctypes.byref(a))


def mlstm_dec_fin(f32, a, m, pairs: int):
    _go("launch_mlstm_dec_fin", f32, ctypes.byref(a), ctypes.byref(m), pairs)


def block_out(f32, Wo, o, ldo: int, m, K1: int, x, rows: int, W: int,
              mult: float):
    _go("launch_block_out", f32, _ptr(Wo), _ptr(o), ldo, ctypes.byref(m), K1,
        _ptr(x), rows, W, mult)


def moe_rows(f32, m, s, y, x, rows: int, mult: float):
    _go("launch_moe_rows", f32, ctypes.byref(m), ctypes.byref(s), _ptr(y),
        _ptr(x), rows, mult)
