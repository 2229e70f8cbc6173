// gqa_attn.hip — grouped-query attention over a paged cache, without
// rotation: RMS norm over the whole query and key projections; as options
// a query factor per position, a sigmoid gate per output element, chunks
// (a token sees the earlier ones of its own chunk of positions), a bias by
// head and distance, a sink per head in the softmax.  Where values are the
// projected keys ahead of their norm, ov is ok.
//
// Page p of a sequence holds positions 64p .. 64p+63, per key/value head as
//   K [64, DP]   a key per row, zero-padded from dim to DP
//   V [VP, 64]   transposed, the keys of each 32 in the order in which the
//                scores leave the MFMA (see v_place), so a lane's operand
//                of the value product is one contiguous piece of a row
// Scores are S^T = K Q^T (a query's statistics stay in the lanes of its
// column), the output is O^T = V^T P^T.  A query tile is 16 (token, head)
// pairs that share a key/value head.
#include "attn_split.h"
#include "gemm_tile.h"
#include "hybrid.h"
#include "mingru.h"

#define PAGE 64
#define TILE_PAIRS 64        // (token, head) pairs of a block over runs

struct GqaArgs {
  const float* P;            // fp32 projections [rows, ldp], biases added
  const float *qnorm, *knorm;   // [H*d], [G*d]
  const float* temp;         // query factor per position, nullable
  const float* bias;         // nullable: [H, nbias] by distance, the last entry
                             // for all beyond it; base-2 exponents
  const float* sink;         // nullable: [H], base-2 exponents
  const int *slot, *pos;     // per row
  const int* table;          // [slots, ldt] page numbers
  void *K, *V;               // [pages, G, 64, DP], [pages, G, VP, 64]
  void* q;                   // [rows, H, DP] (runs)
  float *part, *ml;          // split partials [NS, rows*H, VP], [.., 2]
  void* o;                   // [rows, ldo]
  const int *seg_row0, *seg_len, *seg_slot, *seg_pos0;
  const int *tile_seg, *tile_rr0;
  int ldp, oq, ok, ov, og;   // og < 0: no gate
  int H, G, d, vd, DP, VP, ldo, ldt;
  int rows, rbase, NS;       // rows [rbase, rbase+rows) take part
  int chunk, nbias;          // chunk 0: every earlier position is seen
  float eps, scale;
};

// first position that position p sees
DEVINL int first_seen(const GqaArgs& a, int p) {
  return a.chunk ? p - p % a.chunk : 0;
}

// place of key j (0..63) in a row of V: inside each 32, score fragment i,
// lane group g, register r hold key 16i + 4g + r
DEVINL int v_place(int j) {
  return (j & 32) | ((j >> 2) & 3) << 3 | ((j >> 4) & 1) << 2 | (j & 3);
}

DEVINL float sum_squares(const float* p, int n, float* red) {
  float ss = 0.f;
#pragma unroll 4
  for (int i = threadIdx.x; i < n; i += blockDim.x) ss += p[i] * p[i];
  return block_sum(ss, red);
}

// key and value of key/value head g, written to the cache
template <typename T>
DEVINL void write_kv(const GqaArgs& a, const float* p, int page, int at, int g,
                     float rk) {
  T* K = (T*)a.K + (((size_t)page * a.G + g) * PAGE + at) * a.DP;
  const float* k = p + a.ok + g * a.d;
  for (int i = threadIdx.x; i < a.DP; i += blockDim.x)
    K[i] = El<T>::st(i < a.d ? k[i] * rk * a.knorm[g * a.d + i] : 0.f);
  T* V = (T*)a.V + ((size_t)page * a.G + g) * a.VP * PAGE + v_place(at);
  const float* v = p + a.ov + g * a.vd;
  for (int i = threadIdx.x; i < a.vd; i += blockDim.x)
    V[(size_t)i * PAGE] = El<T>::st(v[i]);
}

// ---- runs: normed queries, keys and values -------------------------------
// a block per row for queries and keys; blocks of PREP_ROWS rows for the
// values, since those of neighbouring positions share a line of V
#define PREP_ROWS 8
#define PREP_U 8             // query elements a thread holds
template <typename T>
__global__ void __launch_bounds__(256) k_gqa_prep(GqaArgs a, int vblocks) {
  __shared__ float red[2][4];
  const int tid = threadIdx.x, wave = wave_index(), lane = tid & 63;
  if ((int)blockIdx.x < vblocks) {
    const int i = blockIdx.x * PREP_ROWS + tid % PREP_ROWS;
    if (i >= a.rows) return;
    const size_t r = a.rbase + i;
    const int pos = a.pos[r];
    const size_t page = a.table[(size_t)a.slot[r] * a.ldt + pos / PAGE];
    const float* v = a.P + r * a.ldp + a.ov;
    T* V = (T*)a.V + page * a.G * a.VP * PAGE + v_place(pos % PAGE);
    for (int g = 0; g < a.G; g++, v += a.vd, V += (size_t)a.VP * PAGE)
#pragma unroll 4
      for (int e = tid / PREP_ROWS; e < a.vd; e += 256 / PREP_ROWS)
        V[(size_t)e * PAGE] = El<T>::st(v[e]);
    return;
  }
  const size_t r = a.rbase + blockIdx.x - vblocks;
  const float* p = a.P + r * a.ldp;
  const int pos = a.pos[r], nq = a.H * a.d, nk = a.G * a.d;
  const int sh = 31 - __clz(a.DP);         // DP is a power of two
  const size_t page = a.table[(size_t)a.slot[r] * a.ldt + pos / PAGE];
  float qv[PREP_U], sq = 0.f, sk = 0.f;
#pragma unroll
  for (int u = 0; u < PREP_U; u++) {
    const int i = tid + u * 256;
    qv[u] = i < nq ? p[a.oq + i] : 0.f;
  }
  for (int i = tid; i < nk; i += 256) sk += p[a.ok + i] * p[a.ok + i];
#pragma unroll
  for (int u = 0; u < PREP_U; u++) sq += qv[u] * qv[u];
  for (int i = tid + PREP_U * 256; i < nq; i += 256)
    sq += p[a.oq + i] * p[a.oq + i];
  sq = wave_reduce_sum(sq);
  sk = wave_reduce_sum(sk);
  if (lane == 0) {
    red[0][wave] = sq;
    red[1][wave] = sk;
  }
  __syncthreads();
  sq = red[0][0] + red[0][1] + red[0][2] + red[0][3];
  sk = red[1][0] + red[1][1] + red[1][2] + red[1][3];
  const float rq = (a.temp ? a.temp[pos] : 1.f) / sqrtf(sq / (float)nq + a.eps);
  const float rk = 1.f / sqrtf(sk / (float)nk + a.eps);
  T* q = (T*)a.q + r * a.H * a.DP;
  if (a.d == a.DP) {                       // no padding: elements stay put
#pragma unroll
    for (int u = 0; u < PREP_U; u++) {
      const int i = tid + u * 256;
      if (i < nq) q[i] = El<T>::st(qv[u] * rq * a.qnorm[i]);
    }
    for (int i = tid + PREP_U * 256; i < nq; i += 256)
      q[i] = El<T>::st(p[a.oq + i] * rq * a.qnorm[i]);
  } else {
    for (int e = tid; e < a.H << sh; e += 256) {
      const int h = e >> sh, j = e - (h << sh), s = h * a.d + j;
      q[e] = El<T>::st(j < a.d ? p[a.oq + s] * rq * a.qnorm[s] : 0.f);
    }
  }
  T* K = (T*)a.K + (page * a.G * PAGE + pos % PAGE) * a.DP;
  for (int e = tid; e < a.G << sh; e += 256) {
    const int g = e >> sh, j = e - (g << sh), s = g * a.d + j;
    K[(size_t)g * PAGE * a.DP + j] =
        El<T>::st(j < a.d ? p[a.ok + s] * rk * a.knorm[s] : 0.f);
  }
}

// ---- pieces of both attention kernels ------------------------------------
// online softmax of a wave: sv[N] are scores (base 2) of this lane's keys
template <int N>
DEVINL float softmax_step(float* sv, float& mrun, float& lrun) {
  float pmax = sv[0];
#pragma unroll
  for (int i = 1; i < N; i++) pmax = fmaxf(pmax, sv[i]);
  pmax = fmaxf(pmax, __shfl_xor(pmax, 16));
  pmax = fmaxf(pmax, __shfl_xor(pmax, 32));
  const float mnew = fmaxf(mrun, pmax);
  const float base = mnew == -INFINITY ? 0.f : mnew;
  const float alpha = __builtin_amdgcn_exp2f(mrun - base);   // 0 while mrun = -inf
  float psum = 0.f;
#pragma unroll
  for (int i = 0; i < N; i++) {
    sv[i] = __builtin_amdgcn_exp2f(sv[i] - base);
    psum += sv[i];
  }
  psum += __shfl_xor(psum, 16);
  psum += __shfl_xor(psum, 32);
  lrun = lrun * alpha + psum;
  mrun = mnew;
  return alpha;
}

// acc += V^T P^T of one 32-key group.  v: this lane's 8 keys of one row of V
// (two 16-byte pieces in fp32)
template <typename T>
DEVINL f4v pv_mma(const f4v* v, const float* p, f4v acc) {
  if constexpr (sizeof(T) == 2) {
    return GemmMma<u16>::mma(v[0], pack_bf16(p), acc);
  } else {
#pragma unroll
    for (int i = 0; i < 8; i++)
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(v[i >> 2][i & 3], p[i], acc,
                                                 0, 0, 0);
    return acc;
  }
}

// zero the values of keys that no token has written yet (key index of
// element i: k0 + 16*(i/4) + 4g + i%4); they may hold anything
template <typename T>
DEVINL void drop_unwritten(f4v* v, int k0, int g, int kend) {
  if constexpr (sizeof(T) == 2) {
    union { f4v f; u16 h[8]; } o;
    o.f = v[0];
#pragma unroll
    for (int i = 0; i < 8; i++)
      if (k0 + (i >> 2) * 16 + g * 4 + (i & 3) >= kend) o.h[i] = 0;
    v[0] = o.f;
  } else {
#pragma unroll
    for (int i = 0; i < 8; i++)
      if (k0 + (i >> 2) * 16 + g * 4 + (i & 3) >= kend)
        v[i >> 2][i & 3] = 0.f;
  }
}

// ---- single tokens --------------------------------------------------------
// A block takes one row, key/value head and share of the keys: group s of
// 128 keys, then s + NS, ...; its 4 waves take 32 keys each, straight from
// the cache, and merge at the end.  The blocks normalise the query
// themselves; the one whose share ends with the new token writes its key
// and value first.
template <typename T, int DP, int VP>
__global__ void __launch_bounds__(256) k_gqa_token(GqaArgs a) {
  constexpr int SZ = sizeof(T), NC = DP * SZ / 64, ND = VP / 16, VV = SZ / 2;
  constexpr int XS = 32 * VP > 4 * DP * SZ ? 32 * VP : 4 * DP * SZ;
  __shared__ __attribute__((aligned(16))) float xs[XS];
  __shared__ float red[4], ms[4][16], ls[4][16];
  T* qs = (T*)xs;                       // [16][DP], then partials [2][16][VP]
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int qc = lane & 15, g = lane >> 4;
  const int R = a.H / a.G, nqt = (R + 15) / 16;
  const int qt = blockIdx.x % nqt, kv = blockIdx.x / nqt % a.G;
  const int r = blockIdx.x / (nqt * a.G);       // from rbase, which is 0
  const int nq = min(16, R - qt * 16), h0 = kv * R + qt * 16;
  const float* p = a.P + (size_t)r * a.ldp;
  const int pos = a.pos[r], kend = pos + 1;
  const int* pages = a.table + (size_t)a.slot[r] * a.ldt;
  // groups from the first key that is seen
  const int k_lo = first_seen(a, pos), g0 = k_lo / 128;
  const int ngroup = (kend + 127) / 128 - g0, split = blockIdx.y;
  const size_t orow = (size_t)r * a.H + h0;
  const size_t n = (size_t)a.rows * a.H;
  if (split >= ngroup) {
    if (tid < nq) a.ml[(split * n + orow + tid) * 2] = -INFINITY;
    if (tid < nq) a.ml[(split * n + orow + tid) * 2 + 1] = 0.f;
    return;
  }
  const float rq =
      (a.temp ? a.temp[pos] : 1.f) / sqrtf(sum_squares(p + a.oq, a.H * a.d, red) /
                              (float)(a.H * a.d) + a.eps);
  if ((ngroup - 1) % a.NS == split) {
    // blocks of one key/value head (nqt > 1) write the same values
    const float rk =
        1.f / sqrtf(sum_squares(p + a.ok, a.G * a.d, red) /
                        (float)(a.G * a.d) + a.eps);
    write_kv<T>(a, p, pages[pos / PAGE], pos % PAGE, kv, rk);
  }
  for (int i = tid; i < 16 * DP; i += 256) {
    const int c = i / DP, j = i - c * DP, s = (h0 + c) * a.d + j;
    qs[i] = El<T>::st(c < nq && j < a.d ? p[a.oq + s] * rq * a.qnorm[s] : 0.f);
  }
  __syncthreads();              // publishes qs, and the new key to the block
  f4v qf[NC];
#pragma unroll
  for (int c = 0; c < NC; c++)
    qf[c] = ld16((const char*)(qs + qc * DP) + c * 64 + g * 16);
  f4v acc[ND];
#pragma unroll
  for (int d = 0; d < ND; d++) acc[d] = {0.f, 0.f, 0.f, 0.f};
  float mrun = -INFINITY, lrun = 0.f;
  const float sc = a.scale * 1.4426950408889634f;       // base-2 exponents
  const int hq = h0 + min(qc, nq - 1);                  // this lane's head
  if (a.sink && split == 0 && wave == 0) {
    mrun = a.sink[hq];
    lrun = 1.f;
  }
  const float* bias = a.bias ? a.bias + (size_t)hq * a.nbias : nullptr;

  for (int grp = g0 + split; grp < g0 + ngroup; grp += a.NS) {
    const int k0 = grp * 128 + wave * 32;
    if (k0 >= kend) break;
    if (k0 + 32 <= k_lo) continue;
    const size_t pg = (size_t)pages[k0 / PAGE] * a.G + kv;
    const char* K = (const char*)((const T*)a.K +
                                  (pg * PAGE + k0 % PAGE + qc) * DP) + g * 16;
    const char* V = (const char*)((const T*)a.V + (pg * VP + qc) * PAGE +
                                  k0 % PAGE + g * 8);
    f4v kf[2][NC], vf[ND][VV];
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
      for (int c = 0; c < NC; c++)
        kf[i][c] = ld16(K + (size_t)i * 16 * DP * SZ + c * 64);
#pragma unroll
    for (int d = 0; d < ND; d++)
#pragma unroll
      for (int u = 0; u < VV; u++)
        vf[d][u] = ld16(V + (size_t)d * 16 * PAGE * SZ + u * 16);
    float bv[8];
#pragma unroll
    for (int i = 0; i < 8; i++) {
      const int n = pos - (k0 + (i >> 2) * 16 + g * 4 + (i & 3));
      bv[i] = bias ? bias[min(max(n, 0), a.nbias - 1)] : 0.f;
    }
    f4v st[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int c = 0; c < NC; c++)
#pragma unroll
      for (int i = 0; i < 2; i++)
        st[i] = GemmMma<T>::mma(kf[i][c], qf[c], st[i]);
    float sv[8];
#pragma unroll
    for (int i = 0; i < 8; i++) {
      const int key = k0 + (i >> 2) * 16 + g * 4 + (i & 3);
      sv[i] = key < kend && key >= k_lo ? fmaf(st[i >> 2][i & 3], sc, bv[i])
                                        : -INFINITY;
    }
    const float alpha = softmax_step<8>(sv, mrun, lrun);
    if (k0 + 32 > kend)
#pragma unroll
      for (int d = 0; d < ND; d++) drop_unwritten<T>(vf[d], k0, g, kend);
#pragma unroll
    for (int d = 0; d < ND; d++) {
#pragma unroll
      for (int j = 0; j < 4; j++) acc[d][j] *= alpha;
      acc[d] = pv_mma<T>(vf[d], sv, acc[d]);
    }
  }

  // merge the waves
  if (g == 0) {
    ms[wave][qc] = mrun;
    ls[wave][qc] = lrun;
  }
  __syncthreads();              // also: every wave has its query fragments
  float mt = ms[0][qc], lt = 0.f;
#pragma unroll
  for (int w = 1; w < 4; w++) mt = fmaxf(mt, ms[w][qc]);
#pragma unroll
  for (int w = 0; w < 4; w++) lt += exp2f(ms[w][qc] - mt) * ls[w][qc];
  const float mine = exp2f(mrun - mt);          // some wave has seen a key
#pragma unroll
  for (int half = 1; half >= 0; half--) {       // waves 2, 3, then 0, 1
    if (wave >> 1 == half)
#pragma unroll
      for (int d = 0; d < ND; d++) {
        f4v* to = (f4v*)(xs + ((wave & 1) * 16 + qc) * VP + d * 16 + g * 4);
        f4v v = {0.f, 0.f, 0.f, 0.f};
        if (half == 0) v = *to;
#pragma unroll
        for (int j = 0; j < 4; j++) v[j] = fmaf(acc[d][j], mine, v[j]);
        *to = v;
      }
    __syncthreads();
  }
  if (wave == 0 && g == 0 && qc < nq) {
    a.ml[(split * n + orow + qc) * 2] = mt;
    a.ml[(split * n + orow + qc) * 2 + 1] = lt;
  }
  for (int i = tid; i < nq * VP; i += 256)
    a.part[(split * n + orow) * VP + i] = xs[i] + xs[16 * VP + i];
}

// ---- runs -------------------------------------------------------------
// 4 waves of 16 (token, head) pairs over key tiles of KT keys in LDS,
// double-buffered by global_load_lds; 16-byte slots are XOR-swizzled by
// the row, in the source address of the DMA and in the fragment reads.
template <typename T, int DP, int VP, bool BIAS>
__global__ void __launch_bounds__(256) k_gqa_run(GqaArgs a) {
  constexpr int SZ = sizeof(T), NC = DP * SZ / 64, ND = VP / 16, VV = SZ / 2;
  constexpr int KT = 128 / SZ, NG = KT / 32;    // 64 keys in bf16, 32 in fp32
  constexpr int KB = KT * DP * SZ, VB = VP * 128;       // bytes of a tile
  constexpr int SPR = DP * SZ / 16;             // 16-byte slots of a key
  extern __shared__ __attribute__((aligned(16))) char lds[];
  const int tid = threadIdx.x, wave = wave_index(), lane = tid & 63;
  const int qc = lane & 15, g = lane >> 4;
  const int R = a.H / a.G, kv = blockIdx.y;
  const int seg = a.tile_seg[blockIdx.x], rr0 = a.tile_rr0[blockIdx.x];
  const int row0 = a.seg_row0[seg], pos0 = a.seg_pos0[seg];
  const int nrr = a.seg_len[seg] * R;
  const int* pages = a.table + (size_t)a.seg_slot[seg] * a.ldt;
  const int my = rr0 + wave * 16 + qc, myc = min(my, nrr - 1);
  const int tok = myc / R, h = kv * R + myc - tok * R, qpos = pos0 + tok;
  const int kend = pos0 + (min(rr0 + TILE_PAIRS, nrr) - 1) / R + 1;
  const int wlast = pos0 + min(rr0 + wave * 16 + 15, nrr - 1) / R;
  // first keys that this lane's token, the wave's first and the block's see
  const int k_lo = first_seen(a, qpos);
  const int w_lo = first_seen(a, pos0 + min(rr0 + wave * 16, nrr - 1) / R);
  const int t0 = first_seen(a, pos0 + rr0 / R) / KT;
  const int ntile = (kend + KT - 1) / KT;
  const int per = (ntile - t0 + a.NS - 1) / a.NS;
  const int t_lo = t0 + blockIdx.z * per, t_hi = min(ntile, t_lo + per);

  auto stage = [&](int buf, int t) {
    const size_t pg = (size_t)pages[t * KT / PAGE] * a.G + kv;
    const char* K = (const char*)((const T*)a.K +
                                  (pg * PAGE + t * KT % PAGE) * DP);
    const char* V =
        (const char*)((const T*)a.V + pg * VP * PAGE + t * KT % PAGE);
    char* kl = lds + buf * (KB + VB);
#pragma unroll
    for (int i = 0; i < KB / 4096; i++) {
      const int L = (i * 4 + wave) * 64 + lane, row = L / SPR, s = L % SPR;
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) uint32_t*)(
              K + row * (DP * SZ) + ((s ^ (row & 7)) * 16)),
          (__attribute__((address_space(3))) uint32_t*)(
              kl + (i * 4 + wave) * 1024),
          16, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < VB / 4096; i++) {
      const int L = (i * 4 + wave) * 64 + lane, row = L >> 3, s = L & 7;
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) uint32_t*)(
              V + (size_t)row * PAGE * SZ + ((s ^ (row & 7)) * 16)),
          (__attribute__((address_space(3))) uint32_t*)(
              kl + KB + (i * 4 + wave) * 1024),
          16, 0, 0);
    }
  };
  if (t_lo < t_hi) stage(0, t_lo);
  float* bl = (float*)(lds + 2 * (KB + VB));     // the group's biases
  for (int i = tid; i < (BIAS ? R * a.nbias : 0); i += 256)
    bl[i] = a.bias[(size_t)kv * R * a.nbias + i];
  const float* bias = bl + (h - kv * R) * a.nbias;
  f4v qf[NC], acc[ND];
  const char* qp = (const char*)((const T*)a.q +
                                 ((size_t)(row0 + tok) * a.H + h) * DP);
#pragma unroll
  for (int c = 0; c < NC; c++) qf[c] = ld16(qp + c * 64 + g * 16);
#pragma unroll
  for (int d = 0; d < ND; d++) acc[d] = {0.f, 0.f, 0.f, 0.f};
  float mrun = -INFINITY, lrun = 0.f;
  if (a.sink && blockIdx.z == 0) {
    mrun = a.sink[h];
    lrun = 1.f;
  }
  const float sc = a.scale * 1.4426950408889634f;
  __syncthreads();

  int cur = 0;
  for (int t = t_lo; t < t_hi; t++) {
    if (t + 1 < t_hi) stage(cur ^ 1, t + 1);
    const int k0 = t * KT;
    if (k0 <= wlast && k0 + KT > w_lo) {
      const char* kl = lds + cur * (KB + VB);
      const char* vl = kl + KB;
      float sv[8 * NG];
#pragma unroll
      for (int j = 0; j < NG; j++) {
        f4v st[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
        for (int c = 0; c < NC; c++)
#pragma unroll
          for (int i = 0; i < 2; i++) {
            const int row = j * 32 + i * 16 + qc;
            st[i] = GemmMma<T>::mma(
                ld16(kl + row * (DP * SZ) + ((c * 4 + g) ^ (row & 7)) * 16),
                qf[c], st[i]);
          }
#pragma unroll
        for (int i = 0; i < 8; i++) {
          const int n = qpos - (k0 + j * 32 + (i >> 2) * 16 + g * 4 + (i & 3));
          float v = st[i >> 2][i & 3] * sc;
          if constexpr (BIAS) v += bias[min(max(n, 0), a.nbias - 1)];
          sv[j * 8 + i] = n >= 0 && n <= qpos - k_lo ? v : -INFINITY;
        }
      }
      const float alpha = softmax_step<8 * NG>(sv, mrun, lrun);
      if (__any(alpha != 1.f)) {
#pragma unroll
        for (int d = 0; d < ND; d++)
#pragma unroll
          for (int j = 0; j < 4; j++) acc[d][j] *= alpha;
      }
      const bool tail = k0 + KT > kend;
#pragma unroll
      for (int j = 0; j < NG; j++)
#pragma unroll
        for (int d = 0; d < ND; d++) {
          const int row = d * 16 + qc;
          f4v v[VV];
#pragma unroll
          for (int u = 0; u < VV; u++)
            v[u] = ld16(vl + row * 128 +
                        (((j * 4 + g) * VV + u) ^ (row & 7)) * 16);
          if (tail) drop_unwritten<T>(v, k0 + j * 32, g, kend);
          acc[d] = pv_mma<T>(v, sv + j * 8, acc[d]);
        }
    }
    __syncthreads();   // drains the DMA in flight, fences the reads
    cur ^= 1;
  }

  if (my >= nrr) return;
  const size_t r = row0 + tok;
  if (a.NS == 1) {
    const float inv = 1.f / lrun;
    const float* gate =
        a.og < 0 ? nullptr : a.P + r * a.ldp + a.og + h * a.vd;
    T* o = (T*)a.o + r * a.ldo + h * a.vd;
#pragma unroll
    for (int d = 0; d < ND; d++)
#pragma unroll
      for (int j = 0; j < 4; j++) {
        const int i = d * 16 + g * 4 + j;
        if (i < a.vd)
          o[i] = El<T>::st(acc[d][j] * inv * (gate ? sigmoid_f(gate[i]) : 1.f));
      }
  } else {
    const size_t pr = (size_t)blockIdx.z * a.rows * a.H +
                      (r - a.rbase) * a.H + h;
    if (g == 0) {
      a.ml[pr * 2] = mrun;
      a.ml[pr * 2 + 1] = lrun;
    }
    if (t_lo < t_hi) {
      float* op = a.part + pr * VP + g * 4;
#pragma unroll
      for (int d = 0; d < ND; d++) *(f4v*)(op + d * 16) = acc[d];
    }
  }
}

// merge the splits and gate, one block per (row, head); further blocks step
// a gated recurrence that stands beside the attention
template <typename T>
__global__ void __launch_bounds__(256) k_gqa_merge(GqaArgs a, MingruArgs m) {
  __shared__ __attribute__((aligned(16))) float sh[MERGE_LDS];
  const int beside = (int)blockIdx.x - a.rows * a.H;
  if (beside >= 0) {
    mingru_token<T>(m, beside);
    return;
  }
  const int rl = blockIdx.x / a.H, h = blockIdx.x - rl * a.H;
  const size_t r = a.rbase + rl;
  const float* gate = a.og < 0 ? nullptr : a.P + r * a.ldp + a.og + h * a.vd;
  T* o = (T*)a.o + r * a.ldo + h * a.vd;
  merge_splits(a.part, a.ml, (size_t)a.rows * a.H, blockIdx.x, a.NS, a.VP, sh,
               [&](int i, float v) {
                 if (i < a.vd)
                   o[i] = El<T>::st(v * (gate ? sigmoid_f(gate[i]) : 1.f));
               });
}

// ---- launchers ---------------------------------------------------------
static bool bad_shape(const GqaArgs& a) {
  return a.rows < 1 || a.rbase < 0 || a.G < 1 || a.H < 1 || a.H % a.G ||
         a.d < 1 || a.d > a.DP || a.vd < 1 || a.vd > a.VP ||
         a.ldo < a.H * a.vd || a.NS < 1 || a.NS > MAX_SPLITS || a.chunk < 0 ||
         (a.bias && a.nbias < 1);
}

extern "C" hipError_t launch_gqa_prep(int f32, const GqaArgs* a,
                                      hipStream_t s) {
  if (bad_shape(*a) || a->DP & (a->DP - 1)) return hipErrorInvalidValue;
  const int vb = (a->rows + PREP_ROWS - 1) / PREP_ROWS;
  dim3 grid(vb + a->rows);
  if (f32) hipLaunchKernelGGL(k_gqa_prep<float>, grid, dim3(256), 0, s, *a, vb);
  else hipLaunchKernelGGL(k_gqa_prep<u16>, grid, dim3(256), 0, s, *a, vb);
  return hipGetLastError();
}

template <typename T, int DP, int VP>
static hipError_t attn_go(const GqaArgs& a, int tiles, hipStream_t s) {
  if (tiles == 0) {
    const int nqt = (a.H / a.G + 15) / 16;
    hipLaunchKernelGGL((k_gqa_token<T, DP, VP>), dim3(a.rows * a.G * nqt, a.NS),
                       dim3(256), 0, s, a);
  } else {
    size_t lds = 2 * ((128 / sizeof(T)) * DP * sizeof(T) + (size_t)VP * 128);
    if (a.bias) {
      lds += (size_t)(a.H / a.G) * a.nbias * sizeof(float);
      if (lds > 159 * 1024) return hipErrorInvalidValue;
      RAISE_LDS((k_gqa_run<T, DP, VP, true>));
      hipLaunchKernelGGL((k_gqa_run<T, DP, VP, true>), dim3(tiles, a.G, a.NS),
                         dim3(256), lds, s, a);
    } else {
      RAISE_LDS((k_gqa_run<T, DP, VP, false>));
      hipLaunchKernelGGL((k_gqa_run<T, DP, VP, false>), dim3(tiles, a.G, a.NS),
                         dim3(256), lds, s, a);
    }
  }
  return hipGetLastError();
}

template <typename T>
static hipError_t attn(const GqaArgs& a, int tiles, hipStream_t s) {
  if (a.DP == 64 && a.VP == 64) return attn_go<T, 64, 64>(a, tiles, s);
  if (a.DP == 64 && a.VP == 128) return attn_go<T, 64, 128>(a, tiles, s);
  if (a.DP == 128 && a.VP == 64) return attn_go<T, 128, 64>(a, tiles, s);
  if (a.DP == 128 && a.VP == 128) return attn_go<T, 128, 128>(a, tiles, s);
  if (a.DP == 256 && a.VP == 256) return attn_go<T, 256, 256>(a, tiles, s);
  return hipErrorInvalidValue;
}

// rows [0, rows), one token each; partials are left in part/ml
extern "C" hipError_t launch_gqa_token(int f32, const GqaArgs* a,
                                       hipStream_t s) {
  if (bad_shape(*a) || a->rbase) return hipErrorInvalidValue;
  return f32 ? attn<float>(*a, 0, s) : attn<u16>(*a, 0, s);
}

// tiles: query tiles of TILE_PAIRS (token, head of the group) pairs
extern "C" hipError_t launch_gqa_run(int f32, const GqaArgs* a, int tiles,
                                     hipStream_t s) {
  if (bad_shape(*a) || tiles < 1) return hipErrorInvalidValue;
  return f32 ? attn<float>(*a, tiles, s) : attn<u16>(*a, tiles, s);
}

// m (nullable): its single tokens take their step in the same launch
extern "C" hipError_t launch_gqa_merge(int f32, const GqaArgs* a,
                                      const MingruArgs* m, hipStream_t s) {
  if (bad_shape(*a) || (m && (mingru_bad_shape(*m) || m->rows < 1)))
    return hipErrorInvalidValue;
  const MingruArgs side = m ? *m : MingruArgs{};
  dim3 grid(a->rows * a->H + (m ? mingru_token_blocks(side) : 0));
  if (f32)
    hipLaunchKernelGGL(k_gqa_merge<float>, grid, dim3(256), 0, s, *a, side);
  else hipLaunchKernelGGL(k_gqa_merge<u16>, grid, dim3(256), 0, s, *a, side);
  return hipGetLastError();
}
