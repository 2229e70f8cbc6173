// moe.hip — token-grouped routed experts (many rows), experts of a few rows
// as matrix-vector products, and the fused output step of a parallel block.
#include "gemm_tile.h"
#include "hybrid.h"
#include "moe.h"

// logits of the rows; routed inside the gate/up kernel, or ahead of the sort
struct RouteArgs {
  const float* z;           // row r, expert e: z[r*ldz + e*lde]
  int* idx;                 // [rows*K1]
  float* wt;
  int ldz, lde, rows, E, top, extra, scores;
};

DEVINL void route(const RouteArgs& a, int r, int top, int extra, int* idx,
                  float* wt) {
  const float* z = a.z + (size_t)r * a.ldz;
  if (a.E <= 64) route_row<1>(z, a.E, top, extra, idx, wt, a.scores, a.lde);
  else route_row<16>(z, a.E, top, extra, idx, wt, a.scores, a.lde);
}

__global__ void __launch_bounds__(256) k_moe_route(RouteArgs a) {
  const int r = blockIdx.x * 4 + (threadIdx.x >> 6), k1 = a.top + a.extra;
  if (r < a.rows) route(a, r, a.top, a.extra, a.idx + r * k1, a.wt + r * k1);
}

// ---- few rows: gate/up of every pair.  Each block routes its row up to its
// ---- own choice; the first block of a row leaves the choices. -------------
template <typename T>
__global__ void __launch_bounds__(256) k_moe_gu_few(MoeArgs m, RouteArgs a) {
  extern __shared__ __attribute__((aligned(16))) char choice[];   // top numbers, top weights
  int* idx = (int*)choice;
  float* wt = (float*)(choice + a.top * sizeof(int));
  const int p = blockIdx.y, r = p / m.K1, j = p - r * m.K1;
  if (threadIdx.x < 64) {
    if (j == 0 && blockIdx.x == 0)
      route(a, r, a.top, a.extra, a.idx + p, a.wt + p);
    // a softmax needs every chosen logit
    if (j < a.top) route(a, r, a.scores ? j + 1 : a.top, 0, idx, wt);
  }
  __syncthreads();
  const bool shared = j == a.top;
  expert_gu_block<T>(m, p, shared ? m.E : idx[j],
                     m.win && !shared ? wt[j] : 1.f, blockIdx.x);
}

// ---- few rows: x[r] += mult * (Wo o_r + sum_j wt_j Down_{e_j} act_j), or
// ---- (set) x[r] = that; ldo = 0: without Wo ------------------------------
// One wave per output element; block b covers 4 elements of row blockIdx.y.
template <typename T>
__global__ void __launch_bounds__(256)
k_block_out(const T* __restrict__ Wo, const T* __restrict__ o, int ldo,
            MoeArgs m, int K1, float* __restrict__ x, int W, float mult,
            int set) {
  constexpr int V = El<T>::V;
  const int r = blockIdx.y, lane = threadIdx.x & 63;
  const int n = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (n >= W) return;
  float acc = 0.f;
  {
    const T* w = Wo + (size_t)n * ldo;
    const T* xr = o + (size_t)r * ldo;
#pragma unroll 4
    for (int k = lane * V; k < ldo; k += 64 * V)
      acc = dot16<T>(ld16nt(w + k), ld16(xr + k), acc);
  }
  for (int j = 0; j < K1; j++) {
    const int p = r * K1 + j, e = m.idx[p];
    const int ff = e == m.E ? m.ffs : m.ff;
    const T* w = moe_down_base<T>(m, e) + (size_t)n * ff;
    const T* xr = (const T*)m.act + (size_t)p * m.ldact;
    float part = 0.f;
#pragma unroll 2
    for (int k = lane * V; k < ff; k += 64 * V)
      part = dot16<T>(ld16nt(w + k), ld16(xr + k), part);
    acc = fmaf(pair_out(m, p), part, acc);
  }
  acc = wave_reduce_sum(acc);
  if (lane == 0) {
    float* to = x + (size_t)r * W + n;
    *to = (set ? 0.f : *to) + mult * acc;
  }
}

// ---- many rows ----------------------------------------------------------
struct MoeSort {
  int* perm;        // pairs in expert order
  int* tile_e;      // expert of a row tile
  int* tile_row0;   // first position in perm
  int* tile_n;      // rows (0: unused tile)
  int pairs, groups, bm, maxtiles;
};

// one block: histogram, offsets, tile list, scatter
__global__ void __launch_bounds__(1024) k_moe_sort(const int* __restrict__ idx,
                                                   MoeSort a) {
  extern __shared__ int sh[];             // count[G], start[G+1], tile0[G+1]
  int *cnt = sh, *start = sh + a.groups, *tile0 = start + a.groups + 1;
  for (int g = threadIdx.x; g < a.groups; g += 1024) cnt[g] = 0;
  __syncthreads();
  for (int p = threadIdx.x; p < a.pairs; p += 1024) atomicAdd(&cnt[idx[p]], 1);
  __syncthreads();
  if (threadIdx.x == 0) {
    int s = 0, t = 0;
    for (int g = 0; g < a.groups; g++) {
      start[g] = s;
      tile0[g] = t;
      s += cnt[g];
      t += (cnt[g] + a.bm - 1) / a.bm;
    }
    start[a.groups] = s;
    tile0[a.groups] = t;
  }
  __syncthreads();
  for (int g = threadIdx.x; g < a.groups; g += 1024)
    for (int t = tile0[g], k = 0; t < tile0[g + 1] && t < a.maxtiles;
         t++, k += a.bm) {
      a.tile_e[t] = g;
      a.tile_row0[t] = start[g] + k;
      a.tile_n[t] = min(a.bm, start[g + 1] - start[g] - k);
    }
  for (int t = tile0[a.groups] + threadIdx.x; t < a.maxtiles; t += 1024)
    a.tile_n[t] = 0;
  __syncthreads();
  for (int g = threadIdx.x; g < a.groups; g += 1024) cnt[g] = 0;
  __syncthreads();
  for (int p = threadIdx.x; p < a.pairs; p += 1024) {
    int g = idx[p];
    a.perm[start[g] + atomicAdd(&cnt[g], 1)] = p;
  }
}

// gate/up of gathered rows; act rows are in expert order
template <typename T, int BM, int BN>
__global__ void __launch_bounds__(256) k_moe_gu(MoeArgs m, MoeSort s) {
  __shared__ __attribute__((aligned(16))) char lds[gemm_lds_bytes<BM, BN>()];
  const int t = blockIdx.y, nr = s.tile_n[t];
  if (nr == 0) return;
  const int e = s.tile_e[t], p0 = s.tile_row0[t];
  const int ff = e == m.E ? m.ffs : m.ff, bn = blockIdx.x * BN;
  if (bn >= 2 * ff) return;
  const float lim = e == m.E ? m.lims : m.lim;
  const T* W = moe_gu_base<T>(m, e);
  f4v acc[BM / 32][BN / 32];
  gemm_mainloop<BM, BN, T>(
      acc, lds,
      [&](int r) {
        return (const T*)m.h +
               (size_t)(s.perm[p0 + min(r, nr - 1)] / m.K1) * m.ldh;
      },
      [&](int r) { return W + (size_t)min(bn + r, 2 * ff - 1) * m.ldh; }, 0,
      m.ldh / GemmMma<T>::BK);
  float wp[BM / 32][4];
#pragma unroll
  for (int i = 0; i < BM / 32; i++)
#pragma unroll
    for (int r = 0; r < 4; r++)
      wp[i][r] = pair_in(m, s.perm[p0 + min(gemm_row0<BM>(i) + r, nr - 1)]);
#pragma unroll
  for (int i = 0; i < BM / 32; i++)
#pragma unroll
    for (int j = 0; j < BN / 32; j += 2) {
      // fragment columns come as 16 gate rows, then their 16 up rows
      const int col = bn + gemm_col<BN>(j);
      const int f = (col >> 5) * 16 + (col & 15);
#pragma unroll
      for (int r = 0; r < 4; r++) {
        const int row = gemm_row0<BM>(i) + r;
        if (row < nr && f < ff)
          ((T*)m.act)[(size_t)(p0 + row) * m.ldact + f] =
              El<T>::st(glu_act(m.glu, acc[i][j][r] * wp[i][r],
                                acc[i][j + 1][r] * wp[i][r], lim));
      }
    }
}

// down projection back to pair order, as T
template <typename T, int BM, int BN>
__global__ void __launch_bounds__(256) k_moe_down(MoeArgs m, MoeSort s,
                                                  T* __restrict__ y) {
  __shared__ __attribute__((aligned(16))) char lds[gemm_lds_bytes<BM, BN>()];
  const int t = blockIdx.y, nr = s.tile_n[t];
  if (nr == 0) return;
  const int e = s.tile_e[t], p0 = s.tile_row0[t], bn = blockIdx.x * BN;
  const int ff = e == m.E ? m.ffs : m.ff;
  const T* W = moe_down_base<T>(m, e);
  f4v acc[BM / 32][BN / 32];
  gemm_mainloop<BM, BN, T>(
      acc, lds,
      [&](int r) {
        return (const T*)m.act + (size_t)(p0 + min(r, nr - 1)) * m.ldact;
      },
      [&](int r) { return W + (size_t)min(bn + r, m.W - 1) * ff; }, 0,
      ff / GemmMma<T>::BK);
#pragma unroll
  for (int i = 0; i < BM / 32; i++)
#pragma unroll
    for (int r = 0; r < 4; r++) {
      const int row = gemm_row0<BM>(i) + r;
      if (row >= nr) continue;
      T* yr = y + (size_t)s.perm[p0 + row] * m.W;
#pragma unroll
      for (int j = 0; j < BN / 32; j++) {
        const int col = bn + gemm_col<BN>(j);
        if (col < m.W) yr[col] = El<T>::st(acc[i][j][r]);
      }
    }
}

// x[t] += mult * sum_j wt[t, j] * y[t, j], or (set) x[t] = that
template <typename T>
__global__ void __launch_bounds__(256)
k_moe_combine(const T* __restrict__ y, MoeArgs m, float* __restrict__ x,
              int K1, int W, float mult, int set) {
  const int t = blockIdx.y, i = blockIdx.x * 256 + threadIdx.x;
  if (i >= W) return;
  float acc = 0.f;
  for (int j = 0; j < K1; j++)
    acc = fmaf(pair_out(m, t * K1 + j),
               El<T>::ld(y[((size_t)t * K1 + j) * W + i]), acc);
  float* to = x + (size_t)t * W + i;
  *to = (set ? 0.f : *to) + mult * acc;
}

// ---- launchers ------------------------------------------------------------
static bool bad_shape(const MoeArgs& m) {
  return m.ldh % 64 || m.ff % 64 || m.ffs % 64 || m.ldact % 8 ||
         m.ldact < m.ff || m.ldact < m.ffs || m.K1 < 1 || m.E < 1;
}

extern "C" hipError_t launch_block_out(int f32, const void* Wo, const void* o,
                                       int ldo, const MoeArgs* m, int K1,
                                       void* x, int rows, int W, float mult,
                                       int set, hipStream_t s) {
  if (rows < 1 || ldo % 64 || (K1 && bad_shape(*m)))
    return hipErrorInvalidValue;
  dim3 grid((W + 3) / 4, rows);
  if (f32)
    hipLaunchKernelGGL(k_block_out<float>, grid, dim3(256), 0, s,
                       (const float*)Wo, (const float*)o, ldo, *m, K1,
                       (float*)x, W, mult, set);
  else
    hipLaunchKernelGGL(k_block_out<u16>, grid, dim3(256), 0, s,
                       (const u16*)Wo, (const u16*)o, ldo, *m, K1, (float*)x,
                       W, mult, set);
  return hipGetLastError();
}

static bool bad_route(const MoeArgs& m, const RouteArgs& a) {
  return bad_shape(m) || a.rows < 1 || a.E != m.E || a.E > 1024 ||
         a.ldz < 1 || a.lde < 1 || a.top < 1 || a.top > a.E || a.top + a.extra != m.K1 ||
         !a.z || a.idx != m.idx || a.wt != m.wt;
}

// routing + gate/up of rows*K1 pairs
extern "C" hipError_t launch_moe_gu_few(int f32, const MoeArgs* m,
                                        const RouteArgs* a, hipStream_t s) {
  if (bad_route(*m, *a) || a->extra > 1) return hipErrorInvalidValue;
  const int ffm = m->ff > m->ffs ? m->ff : m->ffs;
  dim3 grid((ffm + MOE_FPB - 1) / MOE_FPB, a->rows * m->K1);
  const size_t lds = a->top * (sizeof(int) + sizeof(float));
  if (f32) hipLaunchKernelGGL(k_moe_gu_few<float>, grid, dim3(256), lds, s, *m, *a);
  else hipLaunchKernelGGL(k_moe_gu_few<u16>, grid, dim3(256), lds, s, *m, *a);
  return hipGetLastError();
}

extern "C" hipError_t launch_moe_route(const MoeArgs* m, const RouteArgs* a,
                                       hipStream_t s) {
  if (bad_route(*m, *a)) return hipErrorInvalidValue;
  hipLaunchKernelGGL(k_moe_route, dim3((a->rows + 3) / 4), dim3(256), 0, s, *a);
  return hipGetLastError();
}

template <typename T, int BM>
static void moe_go(const MoeArgs& m, const MoeSort& s, void* y,
                   hipStream_t st) {
  constexpr int BN = BM == 128 ? 128 : 64;
  int ffm = m.ff > m.ffs ? m.ff : m.ffs;
  hipLaunchKernelGGL((k_moe_gu<T, BM, BN>),
                     dim3((2 * ffm + BN - 1) / BN, s.maxtiles), dim3(256), 0,
                     st, m, s);
  hipLaunchKernelGGL((k_moe_down<T, BM, BN>),
                     dim3((m.W + BN - 1) / BN, s.maxtiles), dim3(256), 0, st,
                     m, s, (T*)y);
}

template <typename T>
static hipError_t moe_rows(const MoeArgs& m, const MoeSort& s, void* y,
                           float* x, int rows, float mult, int set,
                           hipStream_t st) {
  if (s.bm == 128) moe_go<T, 128>(m, s, y, st);
  else if (s.bm == 64) moe_go<T, 64>(m, s, y, st);
  else moe_go<T, 32>(m, s, y, st);
  hipLaunchKernelGGL(k_moe_combine<T>, dim3((m.W + 255) / 256, rows),
                     dim3(256), 0, st, (const T*)y, m, x, m.K1, m.W, mult, set);
  return hipGetLastError();
}

// sort + gate/up + down + combine over `rows` tokens
extern "C" hipError_t launch_moe_rows(int f32, const MoeArgs* m,
                                      const MoeSort* s, void* y, void* x,
                                      int rows, float mult, int set,
                                      hipStream_t st) {
  if (bad_shape(*m) || rows < 1 || s->pairs != rows * m->K1 ||
      (s->bm != 32 && s->bm != 64 && s->bm != 128) ||
      s->maxtiles < s->pairs / s->bm + s->groups)
    return hipErrorInvalidValue;
  hipLaunchKernelGGL(k_moe_sort, dim3(1), dim3(1024),
                     (3 * s->groups + 2) * sizeof(int), st, m->idx, *s);
  if (f32) return moe_rows<float>(*m, *s, y, (float*)x, rows, mult, set, st);
  return moe_rows<u16>(*m, *s, y, (float*)x, rows, mult, set, st);
}
