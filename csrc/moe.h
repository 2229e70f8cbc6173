// moe.h — routed experts: argument block and the few-row expert kernels'
// device code, shared by the decode kernels of every mixer.
//
// A (token, choice) pair p = token*K1 + j uses expert idx[p] with weight
// wt[p]; K1 = top (+1 when a shared expert exists: it is expert number E,
// runs for every token with weight 1 and may have its own width and
// limit).  Weights apply to the outputs, or (win) to the inputs of the
// routed experts, which for the bias-free halves is a factor on their
// products.  Gate and up rows are interleaved in groups of 16 (16 gate rows,
// then the 16 up rows of the same hidden units), so one MFMA wave holds
// both halves of the GLU.
#pragma once
#include "hybrid.h"

struct MoeArgs {
  const void* h;            // [rows, ldh] normed input, T
  const void* gu;           // [E][2*ff][ldh] then [2*ffs][ldh]
  const void* down;         // [E][W][ff] then [W][ffs]
  const int* idx;           // [rows*K1]
  const float* wt;          // [rows*K1]
  void* act;                // [rows*K1, ldact] T
  int ldh, ldact, W, E, K1, ff, ffs;   // ff, ffs padded to 64
  int glu, win;             // 1: silu; 1: weights on the inputs
  float lim, lims;
};

// factor of pair p's gate/up products, and of its output
DEVINL float pair_in(const MoeArgs& a, int p) { return a.win ? a.wt[p] : 1.f; }
DEVINL float pair_out(const MoeArgs& a, int p) { return a.win ? 1.f : a.wt[p]; }

DEVINL int gu_row(int f) { return (f >> 4) * 32 + (f & 15); }

template <typename T>
DEVINL const T* moe_gu_base(const MoeArgs& a, int e) {
  return (const T*)a.gu + (size_t)e * 2 * a.ff * a.ldh;   // e == E: shared
}
template <typename T>
DEVINL const T* moe_down_base(const MoeArgs& a, int e) {
  return (const T*)a.down + (size_t)e * a.W * a.ff;
}

#define MOE_FPB 8   // hidden units of a block: 4 waves x 2

// one block: pair p of expert e, hidden units [fb*8, fb*8+8); the products
// with the input come times wp
template <typename T>
DEVINL void expert_gu_block(const MoeArgs& a, int p, int e, float wp, int fb) {
  constexpr int V = El<T>::V;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int ff = e == a.E ? a.ffs : a.ff;
  const int f0 = fb * MOE_FPB + wave * 2;
  if (f0 >= ff) return;
  const float lim = e == a.E ? a.lims : a.lim;
  const T* h = (const T*)a.h + (size_t)(p / a.K1) * a.ldh;
  const T* base = moe_gu_base<T>(a, e);
  const T* w[4];
#pragma unroll
  for (int i = 0; i < 2; i++) {
    w[2 * i] = base + (size_t)gu_row(f0 + i) * a.ldh;
    w[2 * i + 1] = w[2 * i] + (size_t)16 * a.ldh;
  }
  float acc[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
  for (int k = lane * V; k < a.ldh; k += 64 * V) {
    f4v x = ld16(h + k);
#pragma unroll
    for (int i = 0; i < 4; i++) acc[i] = dot16<T>(ld16nt(w[i] + k), x, acc[i]);
  }
#pragma unroll
  for (int i = 0; i < 4; i++) acc[i] = wave_reduce_sum(acc[i]) * wp;
  if (lane < 2)
    ((T*)a.act)[(size_t)p * a.ldact + f0 + lane] = El<T>::st(glu_act(
        a.glu, lane ? acc[2] : acc[0], lane ? acc[3] : acc[1], lim));
}

// the same for a pair that is routed already
template <typename T>
DEVINL void expert_gu_block(const MoeArgs& a, int p, int fb) {
  expert_gu_block<T>(a, p, a.idx[p], pair_in(a, p), fb);
}
