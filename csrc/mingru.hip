// mingru.hip — the gated recurrence of mingru.h.
//
// A run of tokens: chunks of 64 first leave their decay and their state from
// zero; then every chunk folds the ones before it in and goes over its
// tokens again, since reading the projections twice costs less than keeping
// decays and states per token.  Wave w holds tokens 16w .. 16w+15.
#include "mingru.h"

#define CH 64      // chunk length

template <typename T>
__global__ void __launch_bounds__(256) k_mingru_step(MingruArgs a) {
  mingru_token<T>(a, blockIdx.x);
}

// decays and additions of this thread's channel for the wave's 16 tokens, and
// what the 16 do together; tokens beyond the chunk leave things as they are
DEVINL void wave_tokens(const MingruArgs& a, int row0, int len, int ch,
                        float (&dec)[16], float (&add)[16], float& A,
                        float& h) {
  const int t0 = wave_index() * 16;
  float z[16], u[16];
#pragma unroll
  for (int t = 0; t < 16; t++) {
    const float* p = a.P + (size_t)(row0 + min(t0 + t, len - 1)) * a.ldp + ch;
    z[t] = p[a.oz];
    u[t] = p[a.ox];
  }
  A = 1.f;
  h = 0.f;
#pragma unroll
  for (int t = 0; t < 16; t++) {
    dec[t] = 1.f;
    add[t] = 0.f;
    if (t0 + t < len) mingru_gate(z[t], u[t], dec[t], add[t]);
    A *= dec[t];
    h = fmaf(dec[t], h, add[t]);
  }
}

// a run's first chunk starts from the stored state, which it keeps in A
__global__ void __launch_bounds__(256) k_mingru_local(MingruArgs a) {
  __shared__ float endA[4][64], endH[4][64];
  const int lane = threadIdx.x & 63, wave = wave_index(), c = blockIdx.y;
  const int ch = blockIdx.x * 64 + lane, cc = min(ch, a.C - 1);
  const int sg = a.chunk_seg[c], row0 = a.chunk_row0[c];
  const bool first = row0 == a.seg_row0[sg];
  float s = 0.f;
  if (first && a.seg_pos0[sg] > 0) s = a.S[(size_t)a.seg_slot[sg] * a.C + cc];
  float dec[16], add[16], A, h;
  wave_tokens(a, row0, a.chunk_len[c], cc, dec, add, A, h);
  endA[wave][lane] = A;
  endH[wave][lane] = h;
  __syncthreads();
  if (wave || ch >= a.C) return;
  h = fmaf(A, s, h);
#pragma unroll
  for (int w = 1; w < 4; w++) {
    h = fmaf(endA[w][lane], h, endH[w][lane]);
    A *= endA[w][lane];
  }
  a.A[(size_t)c * a.C + ch] = first ? s : A;
  a.h[(size_t)c * a.C + ch] = h;
}

template <typename T>
__global__ void __launch_bounds__(256) k_mingru_out(MingruArgs a) {
  __shared__ float endA[4][64], endH[4][64];
  const int lane = threadIdx.x & 63, wave = wave_index(), c = blockIdx.y;
  const int ch = blockIdx.x * 64 + lane, cc = min(ch, a.C - 1);
  const int sg = a.chunk_seg[c], row0 = a.chunk_row0[c], len = a.chunk_len[c];
  const int seg0 = a.seg_row0[sg], first = c - (row0 - seg0) / CH;
  float dec[16], add[16], A, h, g[16];
  wave_tokens(a, row0, len, cc, dec, add, A, h);
#pragma unroll
  for (int t = 0; t < 16; t++)
    g[t] = a.P[(size_t)(row0 + min(wave * 16 + t, len - 1)) * a.ldp + a.og + cc];
  endA[wave][lane] = A;
  endH[wave][lane] = h;
  float s = (c == first ? a.A : a.h)[(size_t)first * a.C + cc];
#pragma unroll 8
  for (int k = first + 1; k < c; k++)
    s = fmaf(a.A[(size_t)k * a.C + cc], s, a.h[(size_t)k * a.C + cc]);
  __syncthreads();
  for (int w = 0; w < wave; w++) s = fmaf(endA[w][lane], s, endH[w][lane]);
  if (ch >= a.C) return;
#pragma unroll
  for (int t = 0; t < 16; t++) {
    const int tt = wave * 16 + t;
    if (tt >= len) break;
    s = fmaf(dec[t], s, add[t]);
    ((T*)a.out)[(size_t)(row0 + tt) * a.ldo + ch] =
        El<T>::st(s * fast_silu(g[t]));
    if (row0 + tt + 1 == seg0 + a.seg_len[sg])
      a.S[(size_t)a.seg_slot[sg] * a.C + ch] = s;
  }
}

// ---- launchers ------------------------------------------------------------
extern "C" hipError_t launch_mingru_step(int f32, const MingruArgs* a,
                                         hipStream_t s) {
  if (mingru_bad_shape(*a) || a->rows < 1) return hipErrorInvalidValue;
  const dim3 grid(mingru_token_blocks(*a));
  if (f32)
    hipLaunchKernelGGL(k_mingru_step<float>, grid, dim3(256), 0, s, *a);
  else hipLaunchKernelGGL(k_mingru_step<u16>, grid, dim3(256), 0, s, *a);
  return hipGetLastError();
}

extern "C" hipError_t launch_mingru_run(int f32, const MingruArgs* a,
                                        hipStream_t s) {
  if (mingru_bad_shape(*a) || a->nchunk < 1) return hipErrorInvalidValue;
  const dim3 grid((a->C + 63) / 64, a->nchunk);
  hipLaunchKernelGGL(k_mingru_local, grid, dim3(256), 0, s, *a);
  if (f32) hipLaunchKernelGGL(k_mingru_out<float>, grid, dim3(256), 0, s, *a);
  else hipLaunchKernelGGL(k_mingru_out<u16>, grid, dim3(256), 0, s, *a);
  return hipGetLastError();
}
