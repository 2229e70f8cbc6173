// mingru.h — gated recurrence whose gate and candidate read the current
// token only.
//
//   z = sigmoid(Z_t),  c = U_t + 1/2 for U_t >= 0, else sigmoid(U_t)
//   S_t = (1 - z) S_{t-1} + z c,   out = S_t silu(G_t)
//
// element by element; Z, U and G are projections with their biases.  State,
// one slot per sequence: S [slot, C], fp32.  A row at position 0 starts from
// zero whatever its slot held.
#pragma once
#include "hybrid.h"

struct MingruArgs {
  const float* P;             // fp32 projections [rows, ldp]
  float* S;                   // [slots, C]
  float *A, *h;               // [chunks, C]: decay and state of whole chunks
  void* out;                  // [rows, ldo]
  const int *slot, *pos;      // per row
  const int *seg_row0, *seg_len, *seg_slot, *seg_pos0;
  const int *chunk_row0, *chunk_len, *chunk_seg;
  int ldp, oz, ox, og, C, ldo, rows, nchunk;   // rows: single tokens
};

DEVINL void mingru_gate(float z, float u, float& dec, float& add) {
  // 1 - sigmoid(z) = sigmoid(-z), without cancellation
  dec = fast_sigmoid(-z);
  add = fast_sigmoid(z) * (u >= 0.f ? u + 0.5f : fast_sigmoid(u));
}

// 256 channels of one row
template <typename T> DEVINL void mingru_token(const MingruArgs& a, int block) {
  const int per = (a.C + 255) / 256, r = block / per;
  const int c = (block - r * per) * 256 + threadIdx.x;
  if (c >= a.C) return;
  const float* p = a.P + (size_t)r * a.ldp + c;
  float* S = a.S + (size_t)a.slot[r] * a.C + c;
  float dec, add;
  mingru_gate(p[a.oz], p[a.ox], dec, add);
  const float s = a.pos[r] == 0 ? add : fmaf(dec, *S, add);
  *S = s;
  ((T*)a.out)[(size_t)r * a.ldo + c] = El<T>::st(s * fast_silu(p[a.og]));
}

inline int mingru_token_blocks(const MingruArgs& a) {
  return a.rows * ((a.C + 255) / 256);
}

inline bool mingru_bad_shape(const MingruArgs& a) {
  return a.C < 1 || a.ldo < a.C || a.rows < 0 || a.nchunk < 0;
}
