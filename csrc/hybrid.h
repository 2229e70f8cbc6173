// hybrid.h — helpers of the mixed-batch kernels.  Activations and weights
// are T = u16 (bf16) or float; the residual stream, projections that feed
// scores or gates, statistics and recurrent state are fp32 for both.
#pragma once
#include "common.h"

template <typename T> struct El;
template <> struct El<u16> {
  static constexpr int V = 8;             // elements of a 16-byte vector
  DEVINL static float ld(u16 v) { return b2f(v); }
  DEVINL static u16 st(float f) { return f2b(f); }
};
template <> struct El<float> {
  static constexpr int V = 4;
  DEVINL static float ld(float v) { return v; }
  DEVINL static float st(float f) { return f; }
};

// acc += dot of two 16-byte vectors of T
template <typename T> DEVINL float dot16(f4v w, f4v x, float acc) {
  if constexpr (sizeof(T) == 2) {
    union { f4v f; u4v_ u; } a, b;
    a.f = w; b.f = x;
#pragma unroll
    for (int i = 0; i < 4; i++) {
      union { uint32_t i; float f; } wl, wh, xl, xh;
      wl.i = a.u[i] << 16; wh.i = a.u[i] & 0xffff0000u;
      xl.i = b.u[i] << 16; xh.i = b.u[i] & 0xffff0000u;
      acc = fmaf(wl.f, xl.f, acc);
      acc = fmaf(wh.f, xh.f, acc);
    }
  } else {
#pragma unroll
    for (int i = 0; i < 4; i++) acc = fmaf(w[i], x[i], acc);
  }
  return acc;
}

// index of this wave in its block, as a scalar
DEVINL int wave_index() {
  return __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
}

// 8 floats -> 8 bf16, to nearest even
typedef __bf16 bf2_ __attribute__((ext_vector_type(2)));
DEVINL f4v pack_bf16(const float* p) {
  union { f4v f; bf2_ h[4]; } o;
#pragma unroll
  for (int i = 0; i < 4; i++)
    o.h[i] = __builtin_convertvector((f2v{p[2 * i], p[2 * i + 1]}), bf2_);
  return o.f;
}

DEVINL f4v ld16(const void* p) { return *(const f4v*)p; }
DEVINL f4v ld16nt(const void* p) {
  return __builtin_nontemporal_load((const f4v*)p);
}

DEVINL float wave_reduce_max(float v) {
#pragma unroll
  for (int m = 1; m < 64; m <<= 1) v = fmaxf(v, __shfl_xor(v, m));
  return v;
}

// orders LDS traffic between the lanes of one wave
DEVINL void wave_sync() {
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
}

// sum over a block of up to 16 waves; red has one float per wave
DEVINL float block_sum(float v, float* red) {
  v = wave_reduce_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float t = 0.f;
  for (int w = 0; w < (int)(blockDim.x >> 6); w++) t += red[w];
  __syncthreads();
  return t;
}

DEVINL float sigmoid_f(float z) { return 1.f / (1.f + expf(-z)); }
DEVINL float logsigmoid_f(float z) {
  return fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
}

// the same from the hardware's exponential, reciprocal and square root, each
// good to an ulp or so, for kernels that are bound by them
DEVINL float fast_exp(float z) {
  return __builtin_amdgcn_exp2f(z * 1.4426950408889634f);
}
DEVINL float fast_sigmoid(float z) {
  return __builtin_amdgcn_rcpf(1.f + fast_exp(-z));
}
DEVINL float fast_silu(float z) { return z * fast_sigmoid(z); }

// GLUs of the routed experts (glu_act): silu(gate)*up, or clamped,
//   g = min(gate, lim), u = clamp(up, -lim, lim), g*sigmoid(1.702 g)*(u+1)
DEVINL float clamped_glu(float gate, float up, float lim) {
  float g = fminf(gate, lim);
  float u = fminf(fmaxf(up, -lim), lim);
  return g * sigmoid_f(1.702f * g) * (u + 1.f);
}

DEVINL float glu_act(int kind, float gate, float up, float lim) {
  return kind ? gate * sigmoid_f(gate) * up : clamped_glu(gate, up, lim);
}

// logits of one row (already fp32, in global or LDS) -> the `top` largest
// and the softmax over them, or with `scores` their sigmoids as they are.
// One wave; E <= 64*EPL.
template <int EPL>
DEVINL void route_row(const float* z, int E, int top, int extra, int* idx,
                      float* wt, int scores = 0, int lde = 1) {
  const int lane = threadIdx.x & 63;
  float v[EPL];
#pragma unroll
  for (int i = 0; i < EPL; i++) {
    int e = lane + i * 64;
    v[i] = e < E ? z[(size_t)e * lde] : -INFINITY;
  }
  float zmax = 0.f, sum = 0.f;
  for (int j = 0; j < top; j++) {
    float bv = -INFINITY;
    int be = 0x7fffffff;
#pragma unroll
    for (int i = 0; i < EPL; i++) {
      int e = lane + i * 64;
      if (e < E && (v[i] > bv || be == 0x7fffffff)) { bv = v[i]; be = e; }
    }
    // largest value, smallest index on ties
#pragma unroll
    for (int m = 1; m < 64; m <<= 1) {
      float ov = __shfl_xor(bv, m);
      int oe = __shfl_xor(be, m);
      if (oe != 0x7fffffff &&
          (be == 0x7fffffff || ov > bv || (ov == bv && oe < be))) {
        bv = ov; be = oe;
      }
    }
    if (be >= E) be = 0;   // NaN logits: stay in range
    if (j == 0) zmax = bv;
    float w = scores ? sigmoid_f(bv) : expf(bv - zmax);
    sum += w;
    if (lane == 0) { idx[j] = be; wt[j] = w; }
#pragma unroll
    for (int i = 0; i < EPL; i++)
      if (lane + i * 64 == be) v[i] = -INFINITY;
  }
  if (lane == 0) {
    if (!scores)
      for (int j = 0; j < top; j++) wt[j] = wt[j] / sum;
    if (extra) { idx[top] = E; wt[top] = 1.f; }   // the shared expert
  }
}

// raise the dynamic LDS limit of a kernel once
#define RAISE_LDS(fn)                                                        \
  do {                                                                       \
    static bool done_ = false;                                               \
    if (!done_) {                                                            \
      hipError_t e_ = hipFuncSetAttribute(                                   \
          (const void*)(fn), hipFuncAttributeMaxDynamicSharedMemorySize,     \
          159 * 1024);                                                       \
      if (e_ != hipSuccess) return e_;                                       \
      done_ = true;                                                          \
    }                                                                        \
  } while (0)
