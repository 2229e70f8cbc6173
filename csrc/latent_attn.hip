// latent_attn.hip — attention over a paged cache of latents.
//
// A cached token is one row [c (rank, zero-padded to RP) | rotated key part
// (padded to RT)]; page p of a sequence holds positions 64p .. 64p+63.
// Scores and outputs stay in latent space: the per-head up-projection of
// the keys is folded into the query (q' = W_uk^T q), so every head reads
// the same rows, and the value up-projection is applied to the attended
// latent.  A query tile is 16 (token, head) pairs of one sequence.  Optional:
// queries that go through a normed latent of their own, a sliding window, a
// sink per head in the softmax, gates per element.
#include "attn_split.h"
#include "gemm_tile.h"
#include "hybrid.h"
#include "moe.h"

#define PAGE 64

struct LatentArgs {
  const float* P;        // fp32 projections [rows, ldp]
  const float* Q;        // few rows: queries [rows, ldq]; head h's unrotated
                         // part at h*qh, its rotated one at oqr + h*qrh
  void* cq;              // normed query latents [rows, QRp]
  const float* qnorm;    // [qrank]
  const float* sink;     // nullable: [H]
  const void* Wuk;       // [H*d, RP]
  const void* Wuv;       // [H*vd, RP]
  const float* cnorm;    // [rank]
  const float *cosT, *sinT;   // [positions, rdims/2]
  const int *slot, *pos; // per row
  const int* table;      // [slots, ldt] page numbers
  void* cache;           // [pages, 64, RP+RT]
  void* qn;              // [rows, H, dp]      (GEMM path)
  void* qa;              // [rows, H, RP+RT]
  float *part, *ml;      // split partials [NS, rows*H, RP], [NS, rows*H, 2]
  void* olat;            // [rows, H, RP]
  void* o;               // [rows, ldo]
  const int *seg_row0, *seg_len, *seg_slot, *seg_pos0;
  const int *tile_seg, *tile_rr0;    // null: one-token segments
  int* ridx;             // router outputs (rows * (rtop + rextra))
  float* rwt;
  int ldp, oq, odkv, og, orouter;
  int H, d, dp, rot, rdims, RT, rank, RP, vd, ldo, ldt;
  int rows, rbase, NS;   // rows [rbase, rbase+rows) take part in the split
  int E, rtop, rextra;
  int ldq, qh, oqr, qrh, qrank, QRp;
  int pairs;             // 1: rotation pairs are (2i, 2i+1), else (i, i+half)
  int win;               // keys a token sees, itself included (0: all)
  int gz, gc;            // gate of (head h, element j): P[og + h*gz + j*gc]
  int written;           // the cache rows are there already
  float eps, scale;
};

// element i (< rot) of the rotated part of v at position p
DEVINL float rotated(const float* v, int i, int dims, const float* c,
                     const float* s, int pairs) {
  const int half = dims >> 1;
  if (i >= dims) return v[i];
  if (pairs) {
    const float o = v[i ^ 1];
    return v[i] * c[i >> 1] + (i & 1 ? o : -o) * s[i >> 1];
  }
  if (i < half) return v[i] * c[i] - v[i + half] * s[i];
  return v[i] * c[i - half] + v[i - half] * s[i - half];
}

// normed latent and rotated key part of one row -> its cache row
template <typename T>
DEVINL void latent_write(const LatentArgs& a, int r, float* red) {
  const float* p = a.P + (size_t)r * a.ldp + a.odkv;
  const int pos = a.pos[r], CS = a.RP + a.RT;
  const int page = a.table[(size_t)a.slot[r] * a.ldt + pos / PAGE];
  T* dst = (T*)a.cache + ((size_t)page * PAGE + pos % PAGE) * CS;
  const float* c = a.cosT + (size_t)pos * (a.rdims >> 1);
  const float* s = a.sinT + (size_t)pos * (a.rdims >> 1);
  float ss = 0.f;
  for (int i = threadIdx.x; i < a.rank; i += blockDim.x) ss += p[i] * p[i];
  const float rn = 1.f / sqrtf(block_sum(ss, red) / (float)a.rank + a.eps);
  for (int i = threadIdx.x; i < CS; i += blockDim.x) {
    float v = 0.f;
    if (i < a.rank) v = p[i] * rn * a.cnorm[i];
    else if (i >= a.RP && i < a.RP + a.rot)
      v = rotated(p + a.rank, i - a.RP, a.rdims, c, s, a.pairs);
    dst[i] = El<T>::st(v);
  }
}

DEVINL void route_from_proj(const float* P, int ldp, int orouter, int E,
                            int top, int extra, int* ridx, float* rwt, int r) {
  const float* z = P + (size_t)r * ldp + orouter;
  const int k1 = top + extra;
  if (E <= 64) route_row<1>(z, E, top, extra, ridx + r * k1, rwt + r * k1);
  else route_row<16>(z, E, top, extra, ridx + r * k1, rwt + r * k1);
}

// ---- many rows: split q, rotate, write the cache, route ----------------
template <typename T>
__global__ void __launch_bounds__(256) k_latent_prep(LatentArgs a) {
  __shared__ float red[4];
  const int r = blockIdx.x;
  const float* q = a.P + (size_t)r * a.ldp + a.oq;
  const int pos = a.pos[r], dq = a.d + a.rot, CS = a.RP + a.RT;
  const float* c = a.cosT + (size_t)pos * (a.rdims >> 1);
  const float* s = a.sinT + (size_t)pos * (a.rdims >> 1);
  T* qn = (T*)a.qn + (size_t)r * a.H * a.dp;
  for (int i = threadIdx.x; i < a.H * a.dp; i += 256) {
    int h = i / a.dp, j = i - h * a.dp;
    qn[i] = El<T>::st(j < a.d ? q[h * dq + j] : 0.f);
  }
  T* qa = (T*)a.qa + (size_t)r * a.H * CS;
  for (int i = threadIdx.x; i < a.H * a.RT; i += 256) {
    int h = i / a.RT, j = i - h * a.RT;
    qa[(size_t)h * CS + a.RP + j] = El<T>::st(
        j < a.rot ? rotated(q + h * dq + a.d, j, a.rdims, c, s, a.pairs) : 0.f);
  }
  latent_write<T>(a, r, red);
  if (a.E > 0 && threadIdx.x < 64)
    route_from_proj(a.P, a.ldp, a.orouter, a.E, a.rtop, a.rextra, a.ridx,
                    a.rwt, r);
}

// ---- normed query latent and cache row (rows of P whose queries are still
// ---- to be projected) ------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256) k_latent_mid(LatentArgs a) {
  __shared__ float red[4];
  const int r = blockIdx.x;
  if (blockIdx.y) {
    latent_write<T>(a, r, red);
    return;
  }
  const float* q = a.P + (size_t)r * a.ldp + a.oq;
  float ss = 0.f;
  for (int i = threadIdx.x; i < a.qrank; i += 256) ss += q[i] * q[i];
  const float rn = 1.f / sqrtf(block_sum(ss, red) / (float)a.qrank + a.eps);
  for (int i = threadIdx.x; i < a.QRp; i += 256)
    ((T*)a.cq)[(size_t)r * a.QRp + i] =
        El<T>::st(i < a.qrank ? q[i] * rn * a.qnorm[i] : 0.f);
}

// ---- few rows: absorb W_uk per (head, latent columns, row); two more
// ---- blocks per row do the cache row and the routing --------------------
#define AB_COLS 128
template <typename T>
__global__ void __launch_bounds__(256) k_latent_dec_prep(LatentArgs a) {
  constexpr int V = El<T>::V;
  __shared__ float red[256 * V];
  const int r = blockIdx.y;
  const int cb = a.RP < AB_COLS ? a.RP : AB_COLS, ncb = a.RP / cb;
  const int h = blockIdx.x / ncb, c0 = (blockIdx.x - h * ncb) * cb;
  if (h >= a.H) {
    if ((int)blockIdx.x == a.H * ncb) {
      if (!a.written) latent_write<T>(a, r, red);
    } else if (threadIdx.x < 64)
      route_from_proj(a.P, a.ldp, a.orouter, a.E, a.rtop, a.rextra, a.ridx,
                      a.rwt, r);
    return;
  }
  const int CS = a.RP + a.RT, tid = threadIdx.x;
  const float* q = a.Q + (size_t)r * a.ldq + (size_t)h * a.qh;
  const float* qr = a.Q + (size_t)r * a.ldq + a.oqr + (size_t)h * a.qrh;
  T* qa = (T*)a.qa + ((size_t)r * a.H + h) * CS;
  // lanes own V latent columns each; the d axis is split over the groups
  const int nv = cb / V, groups = 256 / nv;
  const int grp = tid / nv, cv = tid - grp * nv;
  float acc[V];
#pragma unroll
  for (int j = 0; j < V; j++) acc[j] = 0.f;
  const T* w = (const T*)a.Wuk + (size_t)h * a.d * a.RP + c0 + cv * V;
#pragma unroll 8
  for (int i = grp; i < a.d; i += groups) {
    union { f4v f; T t[V]; } u;
    u.f = ld16(w + (size_t)i * a.RP);
    const float qi = El<T>::ld(El<T>::st(q[i]));
#pragma unroll
    for (int j = 0; j < V; j++) acc[j] = fmaf(qi, El<T>::ld(u.t[j]), acc[j]);
  }
#pragma unroll
  for (int j = 0; j < V; j++) red[grp * cb + cv * V + j] = acc[j];
  __syncthreads();
  for (int i = tid; i < cb; i += 256) {
    float v = 0.f;
    for (int g = 0; g < groups; g++) v += red[g * cb + i];
    qa[c0 + i] = El<T>::st(v);
  }
  if (c0) return;
  const int pos = a.pos[r];
  const float* c = a.cosT + (size_t)pos * (a.rdims >> 1);
  const float* s = a.sinT + (size_t)pos * (a.rdims >> 1);
  for (int j = tid; j < a.RT; j += 256)
    qa[a.RP + j] = El<T>::st(
        j < a.rot ? rotated(qr, j, a.rdims, c, s, a.pairs) : 0.f);
}

// ---- attention --------------------------------------------------------
// S^T = K Q^T keeps a query's statistics in the lanes of its column; the
// PV product accumulates O^T = V^T P^T from the same rows' first RP
// columns.  bf16 keeps a transposed copy of the latent columns in LDS, in
// the key order in which P^T leaves the score MFMA.
#define KT 32

template <typename T, int RP> struct AttnShape {
  static constexpr int NC = RP * sizeof(T) / 64;        // latent chunks
  static constexpr int NRM = 128 * sizeof(T) / 64;      // rotated, at most
  static constexpr int VS = KT + 8;                     // V^T row stride
};

template <typename T>
static size_t attn_lds(int RP, int RT) {
  size_t b = (size_t)KT * ((RP + RT) * sizeof(T) + 16);
  if (sizeof(T) == 2) b += (size_t)RP * (KT + 8) * 2;
  return b;
}

// SHARE: the NW waves hold the same 16 queries and split the latent columns
// of the output (single tokens); otherwise each wave has 16 queries of its
// own.  Where registers allow (AHEAD), the next key tile is loaded while one
// is worked on.
template <typename T, int RP, int NW, bool SHARE>
__global__ void __launch_bounds__(64 * NW) k_latent_attn(LatentArgs a) {
  constexpr bool AHEAD = sizeof(T) == 2;
  using Sh = AttnShape<T, RP>;
  constexpr int QW = SHARE ? 1 : NW;                    // query groups
  constexpr int ND = SHARE ? RP / 16 / NW : RP / 16;    // output fragments
  constexpr int PF = ((RP + 128) * (int)sizeof(T) / 16 + 4 * NW - 1) / (4 * NW);
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int CS = RP + a.RT;
  const int KB = CS * (int)sizeof(T) + 16;              // K row bytes in LDS
  char* kl = smem;
  u16* vt = (u16*)(smem + (size_t)KT * KB);
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int qc = lane & 15, g = lane >> 4;
  const int d0 = SHARE ? wave * ND : 0;
  int seg, rr0;
  if (a.tile_seg) {
    seg = a.tile_seg[blockIdx.x];
    rr0 = a.tile_rr0[blockIdx.x];
  } else {
    const int nth = (a.H + 16 * QW - 1) / (16 * QW);
    seg = blockIdx.x / nth;
    rr0 = (blockIdx.x - seg * nth) * 16 * QW;
  }
  const int row0 = a.seg_row0[seg], pos0 = a.seg_pos0[seg];
  const int nrr = a.seg_len[seg] * a.H;
  const int* pages = a.table + (size_t)a.seg_slot[seg] * a.ldt;
  const int my = rr0 + (SHARE ? 0 : wave * 16) + qc;
  const int myc = my < nrr ? my : nrr - 1;
  const int qpos = pos0 + myc / a.H;
  const int last = min(rr0 + 16 * QW, nrr) - 1;
  const int kend = pos0 + last / a.H + 1;               // keys [0, kend)
  // key tiles of this split, from the first one that the first query sees
  const int tbeg = a.win ? max(0, pos0 + rr0 / a.H - a.win + 1) / KT : 0;
  const int tend = (kend + KT - 1) / KT;
  const int per = (tend - tbeg + a.NS - 1) / a.NS;
  const int t_lo = tbeg + blockIdx.y * per, t_hi = min(tend, t_lo + per);
  const int before = a.win ? qpos - a.win : -1;         // keys this one hides

  // loading: lanes take 16 row pairs x 16-byte columns
  const int kp = tid & 15, cv0 = tid >> 4;
  const int nvec = CS * (int)sizeof(T) / 16;
  const int vpos = (kp < 8 ? (kp >> 1) * 8 : ((kp - 8) >> 1) * 8 + 4) +
                   (kp & 1) * 2;
  f4v p0[PF], p1[PF];
  auto fetch = [&](int t) {
    const int k0 = t * KT;
    // rows past kend are stale or unwritten: read a valid row instead (the
    // mask removes its score, and the value must stay finite)
    const int nk = min(KT, kend - k0);
    const char* src = (const char*)a.cache +
        ((size_t)pages[k0 / PAGE] * PAGE + k0 % PAGE) * CS * sizeof(T);
    const char* s0 = src + (size_t)min(2 * kp, nk - 1) * CS * sizeof(T);
    const char* s1 = src + (size_t)min(2 * kp + 1, nk - 1) * CS * sizeof(T);
#pragma unroll
    for (int i = 0; i < PF; i++) {
      const int cv = cv0 + i * NW * 4;
      if (cv < nvec) {
        p0[i] = ld16(s0 + cv * 16);
        p1[i] = ld16(s1 + cv * 16);
      }
    }
  };
  if (AHEAD && t_lo < t_hi) fetch(t_lo);

  f4v qf[Sh::NC + Sh::NRM];
  const int NR = a.RT * (int)sizeof(T) / 64;
  {
    const char* qp = (const char*)a.qa +
                     ((size_t)row0 * a.H + myc) * CS * sizeof(T) + g * 16;
#pragma unroll
    for (int c = 0; c < Sh::NC; c++) qf[c] = ld16(qp + c * 64);
#pragma unroll
    for (int c = 0; c < Sh::NRM; c++)
      if (c < NR) qf[Sh::NC + c] = ld16(qp + (Sh::NC + c) * 64);
  }
  f4v acc[ND];
#pragma unroll
  for (int d = 0; d < ND; d++) acc[d] = {0.f, 0.f, 0.f, 0.f};
  float mrun = -INFINITY, lrun = 0.f;
  if (a.sink && blockIdx.y == 0) {      // a score without a value
    mrun = a.sink[myc % a.H] * 1.4426950408889634f;
    lrun = 1.f;
  }
  const float sc = a.scale * 1.4426950408889634f;       // base-2 exponents

  for (int t = t_lo; t < t_hi; t++) {
    const int k0 = t * KT;
    if (!AHEAD) fetch(t);
    if (t > t_lo) __syncthreads();
#pragma unroll
    for (int i = 0; i < PF; i++) {
      const int cv = cv0 + i * NW * 4;
      if (cv < nvec) {
        *(f4v*)(kl + (2 * kp) * KB + cv * 16) = p0[i];
        *(f4v*)(kl + (2 * kp + 1) * KB + cv * 16) = p1[i];
        if (sizeof(T) == 2 && cv * 8 < RP) {
          union { f4v f; uint32_t u[4]; } a0, a1;
          a0.f = p0[i]; a1.f = p1[i];
#pragma unroll
          for (int j = 0; j < 4; j++) {
            *(uint32_t*)(vt + (cv * 8 + 2 * j) * Sh::VS + vpos) =
                (a0.u[j] & 0xffffu) | (a1.u[j] << 16);
            *(uint32_t*)(vt + (cv * 8 + 2 * j + 1) * Sh::VS + vpos) =
                (a0.u[j] >> 16) | (a1.u[j] & 0xffff0000u);
          }
        }
      }
    }
    __syncthreads();
    if (AHEAD && t + 1 < t_hi) fetch(t + 1);

    f4v st[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
    const char* kr = kl + qc * KB + g * 16;
#pragma unroll
    for (int c = 0; c < Sh::NC; c++)
#pragma unroll
      for (int i = 0; i < 2; i++)
        st[i] = GemmMma<T>::mma(ld16(kr + i * 16 * KB + c * 64), qf[c], st[i]);
#pragma unroll
    for (int c = 0; c < Sh::NRM; c++)
      if (c < NR)
#pragma unroll
        for (int i = 0; i < 2; i++)
          st[i] = GemmMma<T>::mma(ld16(kr + i * 16 * KB + (Sh::NC + c) * 64),
                                  qf[Sh::NC + c], st[i]);
    float sv[8], pmax = -INFINITY;
#pragma unroll
    for (int i = 0; i < 8; i++) {
      const int key = k0 + (i >> 2) * 16 + g * 4 + (i & 3);
      sv[i] = key <= qpos && key > before ? st[i >> 2][i & 3] * sc : -INFINITY;
      pmax = fmaxf(pmax, sv[i]);
    }
    pmax = fmaxf(pmax, __shfl_xor(pmax, 16));
    pmax = fmaxf(pmax, __shfl_xor(pmax, 32));
    const float mnew = fmaxf(mrun, pmax);
    const float base = mnew == -INFINITY ? 0.f : mnew;
    const float alpha = exp2f(mrun - base);             // 0 while mrun = -inf
    float psum = 0.f;
#pragma unroll
    for (int i = 0; i < 8; i++) {
      sv[i] = exp2f(sv[i] - base);
      psum += sv[i];
    }
    psum += __shfl_xor(psum, 16);
    psum += __shfl_xor(psum, 32);
    lrun = lrun * alpha + psum;
    mrun = mnew;
    if (__any(alpha != 1.f)) {
#pragma unroll
      for (int d = 0; d < ND; d++)
#pragma unroll
        for (int j = 0; j < 4; j++) acc[d][j] *= alpha;
    }
    if constexpr (sizeof(T) == 2) {
      union { f4v f; u16 h[8]; } p;
#pragma unroll
      for (int i = 0; i < 8; i++) p.h[i] = f2b(sv[i]);
#pragma unroll
      for (int d = 0; d < ND; d++)
        acc[d] = GemmMma<u16>::mma(
            ld16(vt + ((d0 + d) * 16 + qc) * Sh::VS + g * 8), p.f, acc[d]);
    } else {
#pragma unroll
      for (int d = 0; d < ND; d++)
#pragma unroll
        for (int i = 0; i < 8; i++)
          acc[d] = __builtin_amdgcn_mfma_f32_16x16x4f32(
              *(const float*)(kl + ((i >> 2) * 16 + g * 4 + (i & 3)) * KB +
                              ((d0 + d) * 16 + qc) * 4),
              sv[i], acc[d], 0, 0, 0);
    }
  }

  if (my >= nrr) return;
  const size_t orow = (size_t)row0 * a.H + my;
  if (a.NS == 1) {
    const float inv = 1.f / lrun;
    T* op = (T*)a.olat + orow * RP + d0 * 16 + g * 4;
#pragma unroll
    for (int d = 0; d < ND; d++) {
      union { T t[4]; uint64_t u; f4v f; } v;
#pragma unroll
      for (int j = 0; j < 4; j++) v.t[j] = El<T>::st(acc[d][j] * inv);
      if constexpr (sizeof(T) == 2) *(uint64_t*)(op + d * 16) = v.u;
      else *(f4v*)(op + d * 16) = v.f;
    }
  } else {
    const size_t pr =
        ((size_t)blockIdx.y * a.rows + row0 - a.rbase) * a.H + my;
    if (g == 0 && (!SHARE || wave == 0)) {
      a.ml[pr * 2] = mrun;
      a.ml[pr * 2 + 1] = lrun;
    }
    if (t_lo < t_hi) {
      float* op = a.part + pr * RP + d0 * 16 + g * 4;
#pragma unroll
      for (int d = 0; d < ND; d++) *(f4v*)(op + d * 16) = acc[d];
    }
  }
}

// merged latent of one (row, head) -> dst (as T)
template <typename T>
DEVINL void latent_merge(const LatentArgs& a, size_t orow, T* dst, float* sh) {
  merge_splits(a.part, a.ml, (size_t)a.rows * a.H, orow, a.NS, a.RP, sh,
               [&](int i, float v) { dst[i] = El<T>::st(v); });
}

template <typename T>
__global__ void __launch_bounds__(256) k_latent_merge(LatentArgs a) {
  __shared__ __attribute__((aligned(16))) float sh[MERGE_LDS];
  latent_merge<T>(a, blockIdx.x,
                  (T*)a.olat + ((size_t)a.rbase * a.H + blockIdx.x) * a.RP,
                  sh);
}

// ---- few rows: merge + value up-projection + gate, in `nub` blocks per
// ---- (row, head); the experts' gate/up halves run beside it ------------
#define UVW 8      // outputs of a wave at a time
template <typename T>
__global__ void __launch_bounds__(256) k_latent_dec_fin(LatentArgs a, int nub,
                                                        MoeArgs m, int fblocks) {
  __shared__ __attribute__((aligned(16))) T ol[512];
  __shared__ __attribute__((aligned(16))) float sh[MERGE_LDS];
  const int nmix = a.rows * a.H * nub;
  if ((int)blockIdx.x >= nmix) {
    const int b = blockIdx.x - nmix;
    expert_gu_block<T>(m, b / fblocks, b % fblocks);
    return;
  }
  constexpr int V = El<T>::V;
  const int rh = blockIdx.x / nub, ub = blockIdx.x - rh * nub;
  const int r = rh / a.H, h = rh - r * a.H;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int nv = a.RP / V;                  // 16-byte vectors of a row
  const T* wb = (const T*)a.Wuv + (size_t)h * a.vd * a.RP;
  T* o = (T*)a.o + (size_t)r * a.ldo + h * a.vd;
  int j0 = (ub * 4 + wave) * UVW;
  f4v w[UVW];                               // on its way during the merge
  auto slab = [&](int k) {
#pragma unroll
    for (int i = 0; i < UVW; i++)
      w[i] = k < nv ? ld16(wb + (size_t)min(j0 + i, a.vd - 1) * a.RP + k * V)
                    : f4v{0.f, 0.f, 0.f, 0.f};
  };
  slab(lane);
  latent_merge<T>(a, rh, ol, sh);
  __syncthreads();
  const float* gate = a.P + (size_t)r * a.ldp + a.og + h * a.gz;
  for (int first = 1; j0 < a.vd; j0 += nub * 4 * UVW, first = 0) {
    float acc[UVW], out = 0.f;
    const bool mine = lane < UVW && j0 + lane < a.vd;
    const float gt = mine ? sigmoid_f(gate[(j0 + lane) * a.gc]) : 0.f;
#pragma unroll
    for (int i = 0; i < UVW; i++) acc[i] = 0.f;
    for (int k = lane; k < nv; k += 64) {
      if (!first || k != lane) slab(k);
      f4v x = ld16(ol + k * V);
#pragma unroll
      for (int i = 0; i < UVW; i++) acc[i] = dot16<T>(w[i], x, acc[i]);
    }
#pragma unroll
    for (int i = 0; i < UVW; i++) {
      float v = wave_reduce_sum(acc[i]);
      if (lane == i) out = v;
    }
    if (mine) o[j0 + lane] = El<T>::st(out * gt);
  }
}

// ---- launchers ---------------------------------------------------------
static bool bad_shape(const LatentArgs& a) {
  return a.rows < 1 || a.H < 1 || a.RT % 32 || a.RT < a.rot || a.RT > 128 ||
         a.RP < a.rank || a.rdims > a.rot || a.rdims % 2 || a.NS < 1 ||
         a.NS > MAX_SPLITS || a.E > 1024 || (a.E > 0 && a.rtop > a.E) || a.dp % 64 ||
         a.dp < a.d || a.win < 0;
}

extern "C" hipError_t launch_latent_prep(int f32, const LatentArgs* a,
                                         hipStream_t s) {
  if (bad_shape(*a)) return hipErrorInvalidValue;
  if (f32) hipLaunchKernelGGL(k_latent_prep<float>, dim3(a->rows), dim3(256), 0, s, *a);
  else hipLaunchKernelGGL(k_latent_prep<u16>, dim3(a->rows), dim3(256), 0, s, *a);
  return hipGetLastError();
}

extern "C" hipError_t launch_latent_mid(int f32, const LatentArgs* a,
                                        hipStream_t s) {
  if (bad_shape(*a) || a->qrank < 1 || a->QRp < a->qrank || !a->cq ||
      !a->qnorm)
    return hipErrorInvalidValue;
  if (f32) hipLaunchKernelGGL(k_latent_mid<float>, dim3(a->rows, 2), dim3(256), 0, s, *a);
  else hipLaunchKernelGGL(k_latent_mid<u16>, dim3(a->rows, 2), dim3(256), 0, s, *a);
  return hipGetLastError();
}

extern "C" hipError_t launch_latent_dec_prep(int f32, const LatentArgs* a,
                                             hipStream_t s) {
  if (bad_shape(*a) || a->RP > 512 || !a->Q) return hipErrorInvalidValue;
  const int cb = a->RP < AB_COLS ? a->RP : AB_COLS;
  if (a->RP % cb) return hipErrorInvalidValue;
  // the last head's blocks: cache row, then routing (RP / cb may be 1)
  dim3 grid(a->H * (a->RP / cb) + (a->E > 0 ? 2 : 1), a->rows);
  if (f32) hipLaunchKernelGGL(k_latent_dec_prep<float>, grid, dim3(256), 0, s, *a);
  else hipLaunchKernelGGL(k_latent_dec_prep<u16>, grid, dim3(256), 0, s, *a);
  return hipGetLastError();
}

template <typename T, int RP>
static hipError_t attn_go(const LatentArgs& a, int share, int tiles,
                          hipStream_t s) {
  size_t lds = attn_lds<T>(RP, a.RT);
  dim3 grid(tiles, a.NS);
  if (share) {
    RAISE_LDS((k_latent_attn<T, RP, 4, true>));
    hipLaunchKernelGGL((k_latent_attn<T, RP, 4, true>), grid, dim3(256), lds,
                       s, a);
  } else {
    RAISE_LDS((k_latent_attn<T, RP, 4, false>));
    hipLaunchKernelGGL((k_latent_attn<T, RP, 4, false>), grid, dim3(256), lds,
                       s, a);
  }
  return hipGetLastError();
}

template <typename T>
static hipError_t attn_rp(const LatentArgs& a, int share, int tiles,
                          hipStream_t s) {
  switch (a.RP) {
    case 64: return attn_go<T, 64>(a, share, tiles, s);
    case 128: return attn_go<T, 128>(a, share, tiles, s);
    case 256: return attn_go<T, 256>(a, share, tiles, s);
    case 384: return attn_go<T, 384>(a, share, tiles, s);
    case 512: return attn_go<T, 512>(a, share, tiles, s);
  }
  return hipErrorInvalidValue;
}

// tiles: query tiles of 16 (share) or 64 (token, head) pairs
extern "C" hipError_t launch_latent_attn(int f32, const LatentArgs* a,
                                         int share, int tiles,
                                         hipStream_t s) {
  if (bad_shape(*a) || tiles < 1) return hipErrorInvalidValue;
  return f32 ? attn_rp<float>(*a, share, tiles, s)
             : attn_rp<u16>(*a, share, tiles, s);
}

extern "C" hipError_t launch_latent_merge(int f32, const LatentArgs* a,
                                          hipStream_t s) {
  if (bad_shape(*a)) return hipErrorInvalidValue;
  dim3 grid(a->rows * a->H);
  if (f32) hipLaunchKernelGGL(k_latent_merge<float>, grid, dim3(256), 0, s, *a);
  else hipLaunchKernelGGL(k_latent_merge<u16>, grid, dim3(256), 0, s, *a);
  return hipGetLastError();
}

extern "C" hipError_t launch_latent_dec_fin(int f32, const LatentArgs* a,
                                            const MoeArgs* m, int pairs,
                                            hipStream_t s) {
  if (bad_shape(*a) || a->RP > 512 || a->NS < 2) return hipErrorInvalidValue;
  int ffm = m->ff > m->ffs ? m->ff : m->ffs;
  int fb = pairs ? (ffm + MOE_FPB - 1) / MOE_FPB : 1;
  int nub = 1;               // spread the heads while there are few of them
  while (nub < 4 && a->rows * a->H * nub < 128 && nub * 4 * UVW < a->vd)
    nub *= 2;
  dim3 grid(a->rows * a->H * nub + pairs * fb);
  if (f32) hipLaunchKernelGGL(k_latent_dec_fin<float>, grid, dim3(256), 0, s, *a, nub, *m, fb);
  else hipLaunchKernelGGL(k_latent_dec_fin<u16>, grid, dim3(256), 0, s, *a, nub, *m, fb);
  return hipGetLastError();
}
