// linear.hip — embedding, norm and linear kernels around an fp32 residual
// stream.  Weights are T = bf16 or float, stored [N, Kp] with the K axis
// zero-padded to a multiple of 64; projections come out in fp32.
#include "gemm_tile.h"
#include "hybrid.h"

// ---- embedding: x = x0 = table[id] * scale ---------------------------
template <typename T>
__global__ void __launch_bounds__(256)
k_embed_rows(const T* __restrict__ table, const int* __restrict__ ids,
             float* __restrict__ x, float* __restrict__ x0, int W, float scale) {
  const int r = blockIdx.x;
  const T* src = table + (size_t)ids[r] * W;
  for (int i = threadIdx.x; i < W; i += 256) {
    float v = El<T>::ld(src[i]) * scale;
    x[(size_t)r * W + i] = v;
    if (x0) x0[(size_t)r * W + i] = v;
  }
}

// ---- per-row RMS norm (g given) or cast of [x | x0] (g null) ----------
// out rows have Kp elements; the padding is written as zero.  `rows`
// (nullable) picks the source row of each output row.
template <typename T>
__global__ void __launch_bounds__(256)
k_norm_rows(const float* __restrict__ x, const float* __restrict__ x0,
            const float* __restrict__ g, const int* __restrict__ rows,
            T* __restrict__ out, int W, int Kp, float eps) {
  __shared__ float red[4];
  const size_t src = rows ? rows[blockIdx.x] : blockIdx.x;
  const float* xr = x + src * W;
  T* o = out + (size_t)blockIdx.x * Kp;
  if (g) {
    float ss = 0.f;
    for (int i = threadIdx.x; i < W; i += 256) ss += xr[i] * xr[i];
    const float rn = 1.f / sqrtf(block_sum(ss, red) / (float)W + eps);
    for (int i = threadIdx.x; i < Kp; i += 256)
      o[i] = i < W ? El<T>::st(xr[i] * rn * g[i]) : El<T>::st(0.f);
  } else {
    const float* x0r = x0 + src * W;
    for (int i = threadIdx.x; i < Kp; i += 256)
      o[i] = El<T>::st(i < W ? xr[i] : i < 2 * W ? x0r[i - W] : 0.f);
  }
}

// ---- few rows: Y[r, n] = W[n] . stage(x_r), one weight stream ---------
// The staging pass normalises (g given) or concatenates [x | x0] into LDS
// as T; block 0 can persist it to hout.  One wave per output row.
// cap > 0: y = cap * tanh(y / cap).
template <typename T, int R>
__global__ void __launch_bounds__(256)
k_lin_rows(const T* __restrict__ Wt, const float* __restrict__ x,
           const float* __restrict__ x0, const float* __restrict__ g,
           const int* __restrict__ rows, T* __restrict__ hout,
           float* __restrict__ y, int N, int W, int Kp, int ldy, float eps,
           float cap) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  constexpr int V = El<T>::V;
  T* xs = (T*)smem;
  float* red = (float*)(smem + (size_t)R * Kp * sizeof(T));   // [4][R]
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  size_t src[R];
#pragma unroll
  for (int r = 0; r < R; r++) src[r] = (size_t)(rows ? rows[r] : r) * W;
  if (g) {
    float ss[R];
#pragma unroll
    for (int r = 0; r < R; r++) ss[r] = 0.f;
    for (int i = threadIdx.x; i < W; i += 256)
#pragma unroll
      for (int r = 0; r < R; r++) {
        float v = x[src[r] + i];
        ss[r] += v * v;
      }
#pragma unroll
    for (int r = 0; r < R; r++) {
      ss[r] = wave_reduce_sum(ss[r]);
      if (lane == 0) red[wave * R + r] = ss[r];
    }
    __syncthreads();
#pragma unroll
    for (int r = 0; r < R; r++)
      ss[r] = 1.f / sqrtf((red[r] + red[R + r] + red[2 * R + r] +
                           red[3 * R + r]) / (float)W + eps);
    for (int i = threadIdx.x; i < Kp; i += 256) {
      float gi = i < W ? g[i] : 0.f;
#pragma unroll
      for (int r = 0; r < R; r++) {
        T v = El<T>::st(i < W ? x[src[r] + i] * ss[r] * gi : 0.f);
        xs[r * Kp + i] = v;
        if (hout && blockIdx.x == 0) hout[(size_t)r * Kp + i] = v;
      }
    }
  } else {
    for (int i = threadIdx.x; i < Kp; i += 256)
#pragma unroll
      for (int r = 0; r < R; r++)
        xs[r * Kp + i] = El<T>::st(i < W ? x[src[r] + i]
                                   : i < 2 * W ? x0[src[r] + i - W] : 0.f);
  }
  __syncthreads();
  for (int n = blockIdx.x * 4 + wave; n < N; n += gridDim.x * 4) {
    const T* wr = Wt + (size_t)n * Kp;
    float acc[R];
#pragma unroll
    for (int r = 0; r < R; r++) acc[r] = 0.f;
    int k = lane * V;
    for (; k + 3 * 64 * V < Kp; k += 4 * 64 * V) {
      f4v w[4];
#pragma unroll
      for (int u = 0; u < 4; u++) w[u] = ld16nt(wr + k + u * 64 * V);
#pragma unroll
      for (int u = 0; u < 4; u++)
#pragma unroll
        for (int r = 0; r < R; r++)
          acc[r] = dot16<T>(w[u], ld16(xs + r * Kp + k + u * 64 * V), acc[r]);
    }
    for (; k < Kp; k += 64 * V) {
      f4v w = ld16nt(wr + k);
#pragma unroll
      for (int r = 0; r < R; r++)
        acc[r] = dot16<T>(w, ld16(xs + r * Kp + k), acc[r]);
    }
#pragma unroll
    for (int r = 0; r < R; r++) {
      float a = wave_reduce_sum(acc[r]);
      if (cap > 0.f) a = cap * tanhf(a / cap);
      if (lane == 0) y[(size_t)r * ldy + n] = a;
    }
  }
}

// ---- many rows: MFMA GEMM ---------------------------------------------
enum { EPI_F32 = 0, EPI_RESADD = 1, EPI_SOFTCAP = 2, EPI_T = 3, EPI_TGATE = 4 };

struct GemmArgs {
  const void *X, *W;
  void* Y;
  const float* gate;        // EPI_TGATE: sigmoid(gate[row*ldg + z])
  int M, N, K, ldx, ldw, ldy, ldg, epi;
  float mult;               // EPI_RESADD multiplier / EPI_SOFTCAP cap
  long xz, wz, yz;          // per-z (head) element offsets
};

template <typename T, int BM, int BN>
__global__ void __launch_bounds__(256) k_gemm(GemmArgs a) {
  __shared__ __attribute__((aligned(16))) char lds[gemm_lds_bytes<BM, BN>()];
  const int bm = blockIdx.y * BM, bn = blockIdx.x * BN, z = blockIdx.z;
  const T* X = (const T*)a.X + (size_t)z * a.xz;
  const T* W = (const T*)a.W + (size_t)z * a.wz;
  f4v acc[BM / 32][BN / 32];
  gemm_mainloop<BM, BN, T>(
      acc, lds,
      [&](int r) { return X + (size_t)min(bm + r, a.M - 1) * a.ldx; },
      [&](int r) { return W + (size_t)min(bn + r, a.N - 1) * a.ldw; }, 0,
      a.K / GemmMma<T>::BK);
#pragma unroll
  for (int i = 0; i < BM / 32; i++)
#pragma unroll
    for (int j = 0; j < BN / 32; j++) {
      const int col = bn + gemm_col<BN>(j);
#pragma unroll
      for (int r = 0; r < 4; r++) {
        const int row = bm + gemm_row0<BM>(i) + r;
        if (row >= a.M || col >= a.N) continue;
        float v = acc[i][j][r];
        size_t o = (size_t)z * a.yz + (size_t)row * a.ldy + col;
        if (a.epi == EPI_F32) ((float*)a.Y)[o] = v;
        else if (a.epi == EPI_RESADD) ((float*)a.Y)[o] += a.mult * v;
        else if (a.epi == EPI_SOFTCAP)
          ((float*)a.Y)[o] = a.mult > 0.f ? a.mult * tanhf(v / a.mult) : v;
        else if (a.epi == EPI_T) ((T*)a.Y)[o] = El<T>::st(v);
        else
          ((T*)a.Y)[o] = El<T>::st(
              v * sigmoid_f(a.gate[(size_t)row * a.ldg + z]));
      }
    }
}

#define BY_TYPE(f32, CALL_BF, CALL_F)                                        \
  do {                                                                       \
    if (f32) { CALL_F; } else { CALL_BF; }                                   \
  } while (0)

extern "C" hipError_t launch_embed_rows(int f32, const void* table,
                                        const void* ids, void* x, void* x0,
                                        int M, int W, float scale,
                                        hipStream_t s) {
  BY_TYPE(f32,
          hipLaunchKernelGGL(k_embed_rows<u16>, dim3(M), dim3(256), 0, s,
                             (const u16*)table, (const int*)ids, (float*)x,
                             (float*)x0, W, scale),
          hipLaunchKernelGGL(k_embed_rows<float>, dim3(M), dim3(256), 0, s,
                             (const float*)table, (const int*)ids, (float*)x,
                             (float*)x0, W, scale));
  return hipGetLastError();
}

extern "C" hipError_t launch_norm_rows(int f32, const void* x, const void* x0,
                                       const void* g, const void* rows,
                                       void* out, int M, int W, int Kp,
                                       float eps, hipStream_t s) {
  BY_TYPE(f32,
          hipLaunchKernelGGL(k_norm_rows<u16>, dim3(M), dim3(256), 0, s,
                             (const float*)x, (const float*)x0,
                             (const float*)g, (const int*)rows, (u16*)out, W,
                             Kp, eps),
          hipLaunchKernelGGL(k_norm_rows<float>, dim3(M), dim3(256), 0, s,
                             (const float*)x, (const float*)x0,
                             (const float*)g, (const int*)rows, (float*)out,
                             W, Kp, eps));
  return hipGetLastError();
}

template <typename T, int R>
static hipError_t lin_rows_r(const T* Wt, const float* x, const float* x0,
                             const float* g, const int* rows, T* hout,
                             float* y, int N, int W, int Kp, int ldy,
                             float eps, float cap, hipStream_t s) {
  size_t lds = (size_t)R * Kp * sizeof(T) + 4 * R * sizeof(float);
  RAISE_LDS((k_lin_rows<T, R>));
  int blocks = (N + 3) / 4;
  if (blocks > 1024) blocks = 1024;
  hipLaunchKernelGGL((k_lin_rows<T, R>), dim3(blocks), dim3(256), lds, s, Wt,
                     x, x0, g, rows, hout, y, N, W, Kp, ldy, eps, cap);
  return hipGetLastError();
}

template <typename T>
static hipError_t lin_rows(const T* Wt, const float* x, const float* x0,
                           const float* g, const int* rows, T* hout, float* y,
                           int M, int N, int W, int Kp, int ldy, float eps,
                           float cap, hipStream_t s) {
  int r0 = 0;
  while (r0 < M) {
    int left = M - r0, R = left >= 8 ? 8 : left >= 4 ? 4 : left >= 2 ? 2 : 1;
    while (R > 1 && (size_t)R * Kp * sizeof(T) > 64 * 1024) R >>= 1;
    if ((size_t)R * Kp * sizeof(T) + 128 > 159 * 1024)
      return hipErrorInvalidValue;
    const float* xr = rows ? x : x + (size_t)r0 * W;
    const float* x0r = (x0 && !rows) ? x0 + (size_t)r0 * W : x0;
    const int* rr = rows ? rows + r0 : nullptr;
    T* hr = hout ? hout + (size_t)r0 * Kp : nullptr;
    float* yr = y + (size_t)r0 * ldy;
    hipError_t e;
    if (R == 8) e = lin_rows_r<T, 8>(Wt, xr, x0r, g, rr, hr, yr, N, W, Kp, ldy, eps, cap, s);
    else if (R == 4) e = lin_rows_r<T, 4>(Wt, xr, x0r, g, rr, hr, yr, N, W, Kp, ldy, eps, cap, s);
    else if (R == 2) e = lin_rows_r<T, 2>(Wt, xr, x0r, g, rr, hr, yr, N, W, Kp, ldy, eps, cap, s);
    else e = lin_rows_r<T, 1>(Wt, xr, x0r, g, rr, hr, yr, N, W, Kp, ldy, eps, cap, s);
    if (e != hipSuccess) return e;
    r0 += R;
  }
  return hipSuccess;
}

extern "C" hipError_t launch_lin_rows(int f32, const void* Wt, const void* x,
                                      const void* x0, const void* g,
                                      const void* rows, void* hout, void* y,
                                      int M, int N, int W, int Kp, int ldy,
                                      float eps, float cap, hipStream_t s) {
  if (f32)
    return lin_rows<float>((const float*)Wt, (const float*)x,
                           (const float*)x0, (const float*)g,
                           (const int*)rows, (float*)hout, (float*)y, M, N, W,
                           Kp, ldy, eps, cap, s);
  return lin_rows<u16>((const u16*)Wt, (const float*)x, (const float*)x0,
                       (const float*)g, (const int*)rows, (u16*)hout,
                       (float*)y, M, N, W, Kp, ldy, eps, cap, s);
}

template <typename T>
static void gemm_go(const GemmArgs& a, int Z, hipStream_t s) {
  long b128 = (long)((a.M + 127) / 128) * ((a.N + 127) / 128) * Z;
  if (a.M <= 32) {
    hipLaunchKernelGGL((k_gemm<T, 32, 64>),
                       dim3((a.N + 63) / 64, (a.M + 31) / 32, Z), dim3(256), 0,
                       s, a);
  } else if (b128 < 300) {
    hipLaunchKernelGGL((k_gemm<T, 64, 64>),
                       dim3((a.N + 63) / 64, (a.M + 63) / 64, Z), dim3(256), 0,
                       s, a);
  } else {
    hipLaunchKernelGGL((k_gemm<T, 128, 128>),
                       dim3((a.N + 127) / 128, (a.M + 127) / 128, Z),
                       dim3(256), 0, s, a);
  }
}

extern "C" hipError_t launch_gemm_rows(int f32, const void* X, const void* W,
                                       void* Y, const void* gate, int M,
                                       int N, int K, int ldx, int ldw,
                                       int ldy, int ldg, int epi, float mult,
                                       int Z, long xz, long wz, long yz,
                                       hipStream_t s) {
  if (M < 1 || N < 1 || K < 64 || K % 64 || ldx < K || ldw < K || Z < 1 ||
      epi < 0 || epi > EPI_TGATE)
    return hipErrorInvalidValue;
  GemmArgs a = {X, W, Y, (const float*)gate, M, N, K, ldx, ldw, ldy, ldg, epi,
                mult, xz, wz, yz};
  if (f32) gemm_go<float>(a, Z, s);
  else gemm_go<u16>(a, Z, s);
  return hipGetLastError();
}
