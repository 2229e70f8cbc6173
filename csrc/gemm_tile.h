// gemm_tile.h — the MFMA main loop that the dense, per-head and grouped
// GEMM kernels share: C[BM,BN] += A[BM,K] * B[BN,K]^T.
//
// T = u16 (bf16, v_mfma_f32_16x16x32_bf16) or float (true fp32,
// v_mfma_f32_16x16x4_f32).  A K-slab is 128 bytes a row for both types
// (64 bf16 or 32 floats), so the staging, the swizzle and the fragment
// addresses are the same; a 16-byte fragment feeds one bf16 MFMA or four
// fp32 ones (the order of k inside a slab is free as long as A and B
// agree on it).
//
// 4 waves (2x2), each a (BM/2)x(BN/2) sub-tile of 16x16 fragments.
// Double-buffered LDS filled by global_load_lds (16 B/lane), one barrier
// per slab.  LDS rows are XOR-swizzled (slot ^= row & 7); the DMA writes
// lane-linear, so the swizzle sits in the per-lane source address and in
// the fragment reads.
//
// `arow` / `brow` map a tile row (clamped by the caller to something
// readable) to its first element, which is how row gathers and
// per-expert weight bases come in.  K must be a multiple of 64.
#pragma once
#include "common.h"

typedef short gt_bf8 __attribute__((ext_vector_type(8)));

template <typename T> struct GemmMma;

template <> struct GemmMma<u16> {
  static constexpr int BK = 64;
  DEVINL static f4v mma(f4v a, f4v b, f4v c) {
    union { f4v f; gt_bf8 h; } ua, ub;
    ua.f = a; ub.f = b;
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(ua.h, ub.h, c, 0, 0, 0);
  }
};

template <> struct GemmMma<float> {
  static constexpr int BK = 32;
  DEVINL static f4v mma(f4v a, f4v b, f4v c) {
#pragma unroll
    for (int j = 0; j < 4; j++)
      c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[j], b[j], c, 0, 0, 0);
    return c;
  }
};

// LDS bytes the main loop needs
template <int BM, int BN>
constexpr int gemm_lds_bytes() { return 2 * (BM + BN) * 128; }

template <int BM, int BN, typename T, class ARow, class BRow>
DEVINL void gemm_mainloop(f4v (&acc)[BM / 32][BN / 32], char* lds,
                          ARow arow, BRow brow, int k_lo, int nt) {
  constexpr int FM = BM / 32, FN = BN / 32;
  constexpr int BK = GemmMma<T>::BK;
  constexpr int VE = 16 / sizeof(T);   // elements of a 16-byte slot
  char* As = lds;
  char* Bs = lds + 2 * BM * 128;
  const int tid = threadIdx.x;
  const int wave = tid >> 6, lane = tid & 63;
  const int wrow = wave >> 1, wcol = wave & 1;
  const int g_r = lane >> 3, g_s = lane & 7;

#pragma unroll
  for (int i = 0; i < FM; i++)
#pragma unroll
    for (int j = 0; j < FN; j++) acc[i][j] = {0.f, 0.f, 0.f, 0.f};

  const T* pa[FM];
  const T* pb[FN];
#pragma unroll
  for (int i = 0; i < FM; i++) {
    int r = wave * (BM / 4) + i * 8 + g_r;
    pa[i] = arow(r) + k_lo + (g_s ^ (r & 7)) * VE;
  }
#pragma unroll
  for (int i = 0; i < FN; i++) {
    int r = wave * (BN / 4) + i * 8 + g_r;
    pb[i] = brow(r) + k_lo + (g_s ^ (r & 7)) * VE;
  }
  auto stage = [&](int buf, int kt) {
#pragma unroll
    for (int i = 0; i < FM; i++)
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) uint32_t*)(
              pa[i] + (size_t)kt * BK),
          (__attribute__((address_space(3))) uint32_t*)(
              As + (buf * BM + wave * (BM / 4) + i * 8) * 128),
          16, 0, 0);
#pragma unroll
    for (int i = 0; i < FN; i++)
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) uint32_t*)(
              pb[i] + (size_t)kt * BK),
          (__attribute__((address_space(3))) uint32_t*)(
              Bs + (buf * BN + wave * (BN / 4) + i * 8) * 128),
          16, 0, 0);
  };

  stage(0, 0);
  __syncthreads();
  const int fr = lane & 15, fk = lane >> 4;
  int cur = 0;
  for (int t = 0; t < nt; t++) {
    if (t + 1 < nt) stage(cur ^ 1, t + 1);
#pragma unroll
    for (int sl = 0; sl < 2; sl++) {
      f4v a[FM], b[FN];
#pragma unroll
      for (int i = 0; i < FM; i++) {
        int ra = wrow * (BM / 2) + i * 16 + fr;
        a[i] = *(const f4v*)(As + (cur * BM + ra) * 128 +
                             ((sl * 4 + fk) ^ (ra & 7)) * 16);
      }
#pragma unroll
      for (int j = 0; j < FN; j++) {
        int rb = wcol * (BN / 2) + j * 16 + fr;
        b[j] = *(const f4v*)(Bs + (cur * BN + rb) * 128 +
                             ((sl * 4 + fk) ^ (rb & 7)) * 16);
      }
#pragma unroll
      for (int i = 0; i < FM; i++)
#pragma unroll
        for (int j = 0; j < FN; j++)
          acc[i][j] = GemmMma<T>::mma(a[i], b[j], acc[i][j]);
    }
    __syncthreads();   // drains the DMA in flight, fences the reads
    cur ^= 1;
  }
}

// C layout: element (row, col) of fragment (i, j), register r
//   row = wrow*BM/2 + i*16 + (lane>>4)*4 + r, col = wcol*BN/2 + j*16 + lane%16
template <int BM> DEVINL int gemm_row0(int i) {
  return ((threadIdx.x >> 6) >> 1) * (BM / 2) + i * 16 +
         ((threadIdx.x & 63) >> 4) * 4;
}
template <int BN> DEVINL int gemm_col(int j) {
  return ((threadIdx.x >> 6) & 1) * (BN / 2) + j * 16 + (threadIdx.x & 15);
}
