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
  const int tid = threadIdx.x;
  T* o = out + (size_t)blockIdx.x * Kp;
  if (g) {
    float ss = 0.f, xv[8], gv[8];       // a short row stays in registers
#pragma unroll
    for (int u = 0; u < 8; u++) {
      const int i = tid + u * 256;
      xv[u] = i < W ? xr[i] : 0.f;
      gv[u] = i < W ? g[i] : 0.f;
      ss += xv[u] * xv[u];
    }
    for (int i = tid + 2048; i < W; i += 256) ss += xr[i] * xr[i];
    const float rn = 1.f / sqrtf(block_sum(ss, red) / (float)W + eps);
#pragma unroll
    for (int u = 0; u < 8; u++) {
      const int i = tid + u * 256;
      if (i < Kp) o[i] = El<T>::st(xv[u] * rn * gv[u]);
    }
    for (int i = tid + 2048; i < Kp; i += 256)
      o[i] = i < W ? El<T>::st(xr[i] * rn * g[i]) : El<T>::st(0.f);
  } else {
    const float* x0r = x0 + src * W;
#pragma unroll 8
    for (int i = tid; i < Kp; i += 256)
      o[i] = El<T>::st(i < W ? xr[i] : i < 2 * W ? x0r[i - W] : 0.f);
  }
}

// ---- one row: y[n] = W[n] . stage(x), one wave per pair of outputs ------
// The staging pass normalises (g given) or concatenates [x | x0] into LDS
// as T; block 0 can persist it to hout.  The first slab of the weights is
// on its way while the row is staged.  cap > 0: y = cap * tanh(y / cap).
template <typename T>
__global__ void __launch_bounds__(256)
k_lin_row(const T* __restrict__ Wt, const float* __restrict__ x,
          const float* __restrict__ x0, const float* __restrict__ g,
          const int* __restrict__ rows, T* __restrict__ hout,
          float* __restrict__ y, int N, int W, int Kp, float eps, float cap) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  __shared__ float red[4];
  constexpr int V = El<T>::V, S = 64 * V;
  T* xs = (T*)smem;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const size_t src = (size_t)(rows ? rows[0] : 0) * W;
  int n = (blockIdx.x * 4 + wave) * 2;
  f4v w[2][4];
  auto slab = [&](int n0, int k0) {
#pragma unroll
    for (int i = 0; i < 2; i++) {
      const T* wr = Wt + (size_t)min(n0 + i, N - 1) * Kp;
#pragma unroll
      for (int u = 0; u < 4; u++) {
        const int k = k0 + u * S + lane * V;
        w[i][u] = k < Kp ? ld16nt(wr + k) : f4v{0.f, 0.f, 0.f, 0.f};
      }
    }
  };
  slab(n, 0);
  if (g) {
    float ss = 0.f, xv[8], gv[8];       // the row stays in registers if short
#pragma unroll
    for (int u = 0; u < 8; u++) {
      const int i = tid + u * 256;
      xv[u] = i < W ? x[src + i] : 0.f;
      gv[u] = i < W ? g[i] : 0.f;
      ss += xv[u] * xv[u];
    }
    for (int i = tid + 2048; i < W; i += 256) {
      float v = x[src + i];
      ss += v * v;
    }
    const float rn = 1.f / sqrtf(block_sum(ss, red) / (float)W + eps);
#pragma unroll
    for (int u = 0; u < 8; u++) {
      const int i = tid + u * 256;
      if (i < Kp) {
        T v = El<T>::st(xv[u] * rn * gv[u]);
        xs[i] = v;
        if (hout && blockIdx.x == 0) hout[i] = v;
      }
    }
    for (int i = tid + 2048; i < Kp; i += 256) {
      T v = El<T>::st(i < W ? x[src + i] * rn * g[i] : 0.f);
      xs[i] = v;
      if (hout && blockIdx.x == 0) hout[i] = v;
    }
  } else {
    for (int i = tid; i < Kp; i += 256)
      xs[i] = El<T>::st(i < W ? x[src + i]
                              : i < 2 * W ? x0[src + i - W] : 0.f);
  }
  __syncthreads();
  for (; n < N; n += gridDim.x * 8) {
    if (n != (int)(blockIdx.x * 4 + wave) * 2) slab(n, 0);
    float acc[2] = {0.f, 0.f};
    for (int k0 = 0; k0 < Kp; k0 += 4 * S) {
      if (k0) slab(n, k0);
#pragma unroll
      for (int u = 0; u < 4; u++) {
        const int k = k0 + u * S + lane * V;
        if (k < Kp) {
          f4v xv = ld16(xs + k);
          acc[0] = dot16<T>(w[0][u], xv, acc[0]);
          acc[1] = dot16<T>(w[1][u], xv, acc[1]);
        }
      }
    }
#pragma unroll
    for (int i = 0; i < 2; i++) {
      float a = wave_reduce_sum(acc[i]);
      if (cap > 0.f) a = cap * tanhf(a / cap);
      if (lane == 0 && n + i < N) y[n + i] = a;
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

template <typename T>
DEVINL void gemm_store(const GemmArgs& a, int z, int row, int col, float v) {
  const size_t o = (size_t)z * a.yz + (size_t)row * a.ldy + col;
  if (a.epi == EPI_F32) ((float*)a.Y)[o] = v;
  else if (a.epi == EPI_RESADD) ((float*)a.Y)[o] += a.mult * v;
  else if (a.epi == EPI_SOFTCAP)
    ((float*)a.Y)[o] = a.mult > 0.f ? a.mult * tanhf(v / a.mult) : v;
  else if (a.epi == EPI_T) ((T*)a.Y)[o] = El<T>::st(v);
  else
    ((T*)a.Y)[o] = El<T>::st(
        v * sigmoid_f(a.gate[(size_t)row * a.ldg + z]));
}

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
        if (row < a.M && col < a.N) gemm_store<T>(a, z, row, col, acc[i][j][r]);
      }
    }
}

// up to 16*MF rows: a tile of 16 outputs per block, K over 8 waves, both
// operands straight from memory (the weights are read once)
template <typename T, int MF>
__global__ void __launch_bounds__(512) k_gemm_skinny(GemmArgs a) {
  __shared__ float red[8 * MF * 256];
  constexpr int U = MF == 1 ? 8 : 4;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int lr = lane & 15, gq = lane >> 4, z = blockIdx.z;
  const int n0 = blockIdx.x * 16, nch = a.K * (int)sizeof(T) / 64;
  const char* wr = (const char*)((const T*)a.W + (size_t)z * a.wz +
                                 (size_t)min(n0 + lr, a.N - 1) * a.ldw) +
                   gq * 16;
  const char* xr[MF];
#pragma unroll
  for (int i = 0; i < MF; i++)
    xr[i] = (const char*)((const T*)a.X + (size_t)z * a.xz +
                          (size_t)min(i * 16 + lr, a.M - 1) * a.ldx) + gq * 16;
  f4v acc[MF];
#pragma unroll
  for (int i = 0; i < MF; i++) acc[i] = {0.f, 0.f, 0.f, 0.f};
  int c = wave;
  for (; c + (U - 1) * 8 < nch; c += U * 8) {
    f4v w[U], xv[U][MF];
#pragma unroll
    for (int u = 0; u < U; u++) {
      w[u] = ld16nt(wr + (size_t)(c + u * 8) * 64);
#pragma unroll
      for (int i = 0; i < MF; i++) xv[u][i] = ld16(xr[i] + (c + u * 8) * 64);
    }
#pragma unroll
    for (int u = 0; u < U; u++)
#pragma unroll
      for (int i = 0; i < MF; i++)
        acc[i] = GemmMma<T>::mma(xv[u][i], w[u], acc[i]);
  }
  for (; c < nch; c += 8) {
    f4v w = ld16nt(wr + (size_t)c * 64);
#pragma unroll
    for (int i = 0; i < MF; i++)
      acc[i] = GemmMma<T>::mma(ld16(xr[i] + c * 64), w, acc[i]);
  }
#pragma unroll
  for (int i = 0; i < MF; i++)
#pragma unroll
    for (int r = 0; r < 4; r++)
      red[(wave * MF + i) * 256 + (gq * 4 + r) * 16 + lr] = acc[i][r];
  __syncthreads();
  for (int e = tid; e < MF * 256; e += 512) {
    float v = 0.f;
#pragma unroll
    for (int u = 0; u < 8; u++) v += red[u * MF * 256 + e];
    const int row = e >> 4, col = n0 + (e & 15);
    if (row < a.M && col < a.N) gemm_store<T>(a, z, row, col, v);
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

template <typename T>
static hipError_t lin_row(const void* Wt, const void* x, const void* x0,
                          const void* g, const void* rows, void* hout, void* y,
                          int N, int W, int Kp, float eps, float cap,
                          hipStream_t s) {
  size_t lds = (size_t)Kp * sizeof(T);
  if (Kp % 64 || lds > 150 * 1024) return hipErrorInvalidValue;
  RAISE_LDS(k_lin_row<T>);
  int blocks = (N + 7) / 8;
  if (blocks > 1024) blocks = 1024;
  hipLaunchKernelGGL(k_lin_row<T>, dim3(blocks), dim3(256), lds, s,
                     (const T*)Wt, (const float*)x, (const float*)x0,
                     (const float*)g, (const int*)rows, (T*)hout, (float*)y,
                     N, W, Kp, eps, cap);
  return hipGetLastError();
}

extern "C" hipError_t launch_lin_row(int f32, const void* Wt, const void* x,
                                     const void* x0, const void* g,
                                     const void* rows, void* hout, void* y,
                                     int N, int W, int Kp, float eps,
                                     float cap, hipStream_t s) {
  return f32 ? lin_row<float>(Wt, x, x0, g, rows, hout, y, N, W, Kp, eps, cap, s)
             : lin_row<u16>(Wt, x, x0, g, rows, hout, y, N, W, Kp, eps, cap, s);
}

template <typename T>
static void gemm_go(const GemmArgs& a, int Z, hipStream_t s) {
  long b128 = (long)((a.M + 127) / 128) * ((a.N + 127) / 128) * Z;
  dim3 sk((a.N + 15) / 16, 1, Z);
  if (a.M <= 16) {
    hipLaunchKernelGGL((k_gemm_skinny<T, 1>), sk, dim3(512), 0, s, a);
  } else if (a.M <= 32) {
    hipLaunchKernelGGL((k_gemm_skinny<T, 2>), sk, dim3(512), 0, s, a);
  } else if (a.M <= 64) {
    hipLaunchKernelGGL((k_gemm_skinny<T, 4>), sk, dim3(512), 0, s, a);
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
