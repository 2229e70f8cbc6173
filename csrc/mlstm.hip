// mlstm.hip — matrix-memory LSTM with an exponential input gate.
//
//   m_t = max(f + m_{t-1}, i)                     (m starts at 0)
//   S_t = e^(f + m_{t-1} - m_t) S_{t-1} + e^(i - m_t) k v^T,  n_t alike
//   o_t = S_t^T q / (max(|n_t . q|, e^-m_t) + 1e-6)
//
// State is fp32, one slot per sequence: S [slot, H, d, vd]; n and m are
// kept once per 64-column tile of vd (every tile's block updates its own
// copy, so no block reads what another one writes).  A row at position 0
// starts from zero state whatever its slot held.
//
// Runs of tokens use the chunkwise form of the same recurrence: with F the
// running sum of f inside a chunk and m0 the maximum before it,
//   m_t = F_t + max(m0, max_{s<=t} (i_s - F_s)),
// token s reaches token t with weight e^(F_t - F_s + i_s - m_t), and the
// state before the chunk with e^(F_t + m0 - m_t); every exponent is <= 0.
// Products run on fp32 MFMA (16x16x4) for both activation types.
#include "hybrid.h"
#include "moe.h"

#define CH 64     // chunk length
#define VT 64     // value columns of a tile

struct MlstmArgs {
  const float* P;             // fp32 projections [rows, ldp]
  const float *ib, *fb;       // gate biases [H]
  const float* norm;          // [H*vd]
  float *S, *n, *m;
  float* o;                   // raw outputs [rows, H*vd]
  void* out;                  // normed and gated [rows, ldo], T
  const int *slot, *pos;      // per row
  const int *seg_row0, *seg_len, *seg_slot, *seg_pos0, *seg_chunk0;
  const int *chunk_row0, *chunk_len;
  float *gF, *gi, *gm;        // [rows, H]: F, i, max of i - F so far
  float* cm0;                 // [chunks, H] maximum before the chunk
  float *U, *un;              // [chunks, H, d, vd], [chunks, H, d]
  int* ridx;
  float* rwt;
  int ldp, oq, ok, ov, og, oi, of, orouter;
  int H, d, vd, nvt, ldo, rows, nseg, nchunk;
  int E, rtop, rextra;
  float cap, eps;
};

DEVINL float gate_i(const MlstmArgs& a, int r, int h) {
  return a.cap * tanhf((a.P[(size_t)r * a.ldp + a.oi + h] + a.ib[h]) / a.cap);
}
DEVINL float gate_f(const MlstmArgs& a, int r, int h) {
  return logsigmoid_f(
      a.cap * tanhf((a.P[(size_t)r * a.ldp + a.of + h] + a.fb[h]) / a.cap));
}

// ---- one token per row ------------------------------------------------
// 16 waves per (head, column tile): a wave's lanes own the 64 columns, the
// rows of S are dealt to the waves.  The first rows are on their way while
// the gates are worked out.
#define SW 16
#define SPRE 8
__global__ void __launch_bounds__(64 * SW) k_mlstm_step(MlstmArgs a) {
  extern __shared__ float sm[];           // q[d], k[d], part[SW*64]
  __shared__ float red[SW];
  const int r = blockIdx.y;
  if ((int)blockIdx.x == a.H * a.nvt) {
    if (threadIdx.x < 64) {
      const float* z = a.P + (size_t)r * a.ldp + a.orouter;
      const int k1 = a.rtop + a.rextra;
      if (a.E <= 64)
        route_row<1>(z, a.E, a.rtop, a.rextra, a.ridx + r * k1, a.rwt + r * k1);
      else
        route_row<16>(z, a.E, a.rtop, a.rextra, a.ridx + r * k1, a.rwt + r * k1);
    }
    return;
  }
  const int h = blockIdx.x / a.nvt, vtile = blockIdx.x - h * a.nvt;
  const int tid = threadIdx.x, c = tid & 63, w = tid >> 6;
  float *qs = sm, *ks = sm + a.d, *part = sm + 2 * a.d;
  const float* p = a.P + (size_t)r * a.ldp;
  const size_t sl = a.slot[r];
  const bool fresh = a.pos[r] == 0;
  const int col = vtile * VT + c;
  const bool live = col < a.vd;
  float* S = a.S + ((sl * a.H + h) * a.d) * (size_t)a.vd + col;
  float pre[SPRE];
#pragma unroll
  for (int u = 0; u < SPRE; u++) {
    const int i = w + u * SW;
    pre[u] = (live && !fresh && i < a.d) ? S[(size_t)i * a.vd] : 0.f;
  }
  const float v = live ? p[a.ov + h * a.vd + col] : 0.f;
  float* np = a.n + ((sl * a.H + h) * a.nvt + vtile) * a.d;
  float* mp = a.m + (sl * a.H + h) * a.nvt + vtile;
  const float m0 = fresh ? 0.f : *mp;
  const float gi = gate_i(a, r, h), gf = gate_f(a, r, h);
  const float m1 = fmaxf(gf + m0, gi);
  const float keep = fresh ? 0.f : expf(gf + m0 - m1), add = expf(gi - m1);
  const float qscale = 1.f / sqrtf((float)a.d);
  float nq = 0.f;
  for (int i = tid; i < a.d; i += 64 * SW) {
    float q = p[a.oq + h * a.d + i] * qscale, k = p[a.ok + h * a.d + i] * add;
    qs[i] = q;
    ks[i] = k;
    float nv = fresh ? k : keep * np[i] + k;
    np[i] = nv;
    nq += nv * q;
  }
  nq = block_sum(nq, red);                 // its barriers publish qs and ks
  float acc = 0.f;
  if (live) {
#pragma unroll
    for (int u = 0; u < SPRE; u++) {
      const int i = w + u * SW;
      if (i < a.d) {
        const float s = keep * pre[u] + ks[i] * v;
        S[(size_t)i * a.vd] = s;
        acc = fmaf(s, qs[i], acc);
      }
    }
#pragma unroll 4
    for (int i = w + SPRE * SW; i < a.d; i += SW) {
      float s = ks[i] * v;
      if (!fresh) s += keep * S[(size_t)i * a.vd];
      S[(size_t)i * a.vd] = s;
      acc = fmaf(s, qs[i], acc);
    }
  }
  part[w * VT + c] = acc;
  __syncthreads();
  if (tid < VT && live) {
    float num = 0.f;
#pragma unroll
    for (int u = 0; u < SW; u++) num += part[u * VT + c];
    a.o[(size_t)r * a.H * a.vd + h * a.vd + col] =
        num / (fmaxf(fabsf(nq), expf(-m1)) + 1e-6f);
  }
  if (tid == 0) *mp = m1;      // read before the barriers above
}

// ---- runs of tokens -----------------------------------------------------
// gates inside a chunk, one wave per (head, chunk): F and the running
// maximum M of i - F; m_t follows once the maximum before the chunk is known
__global__ void __launch_bounds__(64) k_mlstm_gates(MlstmArgs a) {
  const int h = blockIdx.x, c = blockIdx.y, lane = threadIdx.x;
  const int r = a.chunk_row0[c] + lane;
  const bool live = lane < a.chunk_len[c];
  const float gi = live ? gate_i(a, r, h) : 0.f;
  float F = live ? gate_f(a, r, h) : 0.f;
#pragma unroll
  for (int s = 1; s < 64; s <<= 1) {
    float o = __shfl_up(F, s);
    if (lane >= s) F += o;
  }
  float M = live ? gi - F : -INFINITY;
#pragma unroll
  for (int s = 1; s < 64; s <<= 1) {
    float o = __shfl_up(M, s);
    if (lane >= s) M = fmaxf(M, o);
  }
  if (live) {
    a.gF[(size_t)r * a.H + h] = F;
    a.gi[(size_t)r * a.H + h] = gi;
    a.gm[(size_t)r * a.H + h] = M;
  }
}

// m before every chunk, and the new state maximum: one wave per (head,
// segment), 64 chunks at a time.  gM = max(m0, .) + F at a chunk's end.
__global__ void __launch_bounds__(64) k_mlstm_chain(MlstmArgs a) {
  const int h = blockIdx.x, sg = blockIdx.y, lane = threadIdx.x;
  const int c0 = a.seg_chunk0[sg], nc = (a.seg_len[sg] + CH - 1) / CH;
  float* mp = a.m + ((size_t)a.seg_slot[sg] * a.H + h) * a.nvt;
  float m0 = a.seg_pos0[sg] == 0 ? 0.f : mp[0];
  for (int b = 0; b < nc; b += 64) {
    const int n = min(64, nc - b), c = c0 + b + min(lane, n - 1);
    const size_t last =
        (size_t)(a.chunk_row0[c] + a.chunk_len[c] - 1) * a.H + h;
    const float F = a.gF[last], M = a.gm[last];
    float mine = m0;
    for (int k = 0; k < n; k++) {
      if (lane == k) mine = m0;
      m0 = __shfl(F, k) + fmaxf(m0, __shfl(M, k));
    }
    if (lane < n) a.cm0[(size_t)c * a.H + h] = mine;
  }
  for (int i = lane; i < a.nvt; i += 64) mp[i] = m0;
}

// what a chunk adds to the state: U = sum_s w_s k_s v_s^T, un = sum_s w_s k_s
#define LS 68     // LDS row stride of a 64-wide fp32 tile
__global__ void __launch_bounds__(256) k_mlstm_local(MlstmArgs a) {
  __shared__ __attribute__((aligned(16))) float kl[CH * LS], vl[CH * LS];
  __shared__ float wl[CH];
  const int c = blockIdx.y, h = blockIdx.z;
  const int ndt = (a.d + 63) / 64;
  const int vtile = blockIdx.x / ndt, dt = blockIdx.x - vtile * ndt;
  const int row0 = a.chunk_row0[c], len = a.chunk_len[c];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const size_t last = (size_t)(row0 + len - 1) * a.H + h;
  const float Fe = a.gF[last];
  const float me = Fe + fmaxf(a.cm0[(size_t)c * a.H + h], a.gm[last]);
  if (tid < CH) {
    const size_t gx = (size_t)(row0 + min(tid, len - 1)) * a.H + h;
    wl[tid] = tid < len ? expf(Fe - a.gF[gx] + a.gi[gx] - me) : 0.f;
  }
  const int j = tid & 63;
  const bool dl = dt * 64 + j < a.d, vl_ = vtile * VT + j < a.vd;
  const float* pk = a.P + a.ok + h * a.d + dt * 64 + j;
  const float* pv = a.P + a.ov + h * a.vd + vtile * VT + j;
  float kv[16], vv[16];
#pragma unroll
  for (int u = 0; u < 16; u++) {
    const int s = wave + u * 4;
    const size_t ro = (size_t)(row0 + min(s, len - 1)) * a.ldp;
    kv[u] = dl ? pk[ro] : 0.f;
    vv[u] = vl_ ? pv[ro] : 0.f;
  }
  __syncthreads();
#pragma unroll
  for (int u = 0; u < 16; u++) {
    const int s = wave + u * 4;
    kl[s * LS + j] = kv[u] * wl[s];          // 0 past the chunk
    vl[s * LS + j] = vv[u];
  }
  __syncthreads();
  const int lr = lane & 15, g = lane >> 4;
  f4v acc[4];
#pragma unroll
  for (int j = 0; j < 4; j++) acc[j] = {0.f, 0.f, 0.f, 0.f};
  for (int s = 0; s < CH; s += 4) {
    const float av = kl[(s + g) * LS + wave * 16 + lr];
#pragma unroll
    for (int j = 0; j < 4; j++)
      acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(
          av, vl[(s + g) * LS + j * 16 + lr], acc[j], 0, 0, 0);
  }
  float* U = a.U + ((size_t)c * a.H + h) * a.d * a.vd;
#pragma unroll
  for (int j = 0; j < 4; j++)
#pragma unroll
    for (int r = 0; r < 4; r++) {
      const int di = dt * 64 + wave * 16 + g * 4 + r;
      const int vi = vtile * VT + j * 16 + lr;
      if (di < a.d && vi < a.vd) U[(size_t)di * a.vd + vi] = acc[j][r];
    }
  if (vtile == 0 && tid < 64 && dt * 64 + tid < a.d) {
    float s0 = 0.f;
    for (int s = 0; s < CH; s++) s0 += kl[s * LS + tid];
    a.un[((size_t)c * a.H + h) * a.d + dt * 64 + tid] = s0;
  }
}

// carry the state over the chunks; U/un become the state BEFORE each chunk
__global__ void __launch_bounds__(256) k_mlstm_scan(MlstmArgs a) {
  const int h = blockIdx.y, sg = blockIdx.z;
  const int i = blockIdx.x * 256 + threadIdx.x;
  const int dv = a.d * a.vd;
  if (i >= dv + a.d) return;
  const size_t sl = a.seg_slot[sg];
  const int c0 = a.seg_chunk0[sg], nc = (a.seg_len[sg] + CH - 1) / CH;
  const bool isn = i >= dv;
  float* st = isn ? a.n + (sl * a.H + h) * a.nvt * a.d + (i - dv)
                  : a.S + (sl * a.H + h) * (size_t)dv + i;
  float cur = a.seg_pos0[sg] == 0 ? 0.f : *st;
  for (int c = c0; c < c0 + nc; c++) {
    const size_t last =
        (size_t)(a.chunk_row0[c] + a.chunk_len[c] - 1) * a.H + h;
    const float mc = a.cm0[(size_t)c * a.H + h];
    const float keep = expf(mc - fmaxf(mc, a.gm[last]));
    float* u = isn ? a.un + ((size_t)c * a.H + h) * a.d + (i - dv)
                   : a.U + ((size_t)c * a.H + h) * (size_t)dv + i;
    const float add = *u;
    *u = cur;
    cur = keep * cur + add;
  }
  if (isn) {
    for (int t = 0; t < a.nvt; t++) st[(size_t)t * a.d] = cur;
  } else {
    *st = cur;
  }
}

// outputs of a chunk: wave w holds tokens 16w .. 16w+15
__global__ void __launch_bounds__(256) k_mlstm_out(MlstmArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float *ql = sm, *kl = sm + CH * LS, *sl = sm + 2 * CH * LS;
  float *Fl = sm + 3 * CH * LS, *il = Fl + CH, *ml = il + CH, *nl = ml + CH;
  const int vtile = blockIdx.x, c = blockIdx.y, h = blockIdx.z;
  const int row0 = a.chunk_row0[c], len = a.chunk_len[c];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int lr = lane & 15, g = lane >> 4;
  const float m0 = a.cm0[(size_t)c * a.H + h];
  const float qscale = 1.f / sqrtf((float)a.d);
  const float* U = a.U + ((size_t)c * a.H + h) * a.d * a.vd;
  const float* un = a.un + ((size_t)c * a.H + h) * a.d;
  if (tid < CH) {
    const size_t gx = (size_t)(row0 + min(tid, len - 1)) * a.H + h;
    Fl[tid] = a.gF[gx];
    il[tid] = a.gi[gx];
    ml[tid] = a.gF[gx] + fmaxf(m0, a.gm[gx]);
  }
  f4v sc[4], acc[4];
#pragma unroll
  for (int j = 0; j < 4; j++)
    sc[j] = acc[j] = f4v{0.f, 0.f, 0.f, 0.f};
  float nq = 0.f;        // q_t . n before the chunk, a quarter per thread
  for (int d0 = 0; d0 < a.d; d0 += 64) {
    const int j = tid & 63, v = vtile * VT + j;
    const bool dl = d0 + j < a.d, vlive = v < a.vd;
    const float* pq = a.P + a.oq + h * a.d + d0 + j;
    const float* pk = a.P + a.ok + h * a.d + d0 + j;
    float qv[16], kv[16], uv[16];
#pragma unroll
    for (int u = 0; u < 16; u++) {
      const int s = wave + u * 4;            // a token, and a row of U
      const size_t ro = (size_t)(row0 + min(s, len - 1)) * a.ldp;
      qv[u] = dl ? pq[ro] : 0.f;
      kv[u] = dl ? pk[ro] : 0.f;
      uv[u] = (d0 + s < a.d && vlive) ? U[(size_t)(d0 + s) * a.vd + v] : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int u = 0; u < 16; u++) {
      const int s = wave + u * 4;
      ql[s * LS + j] = s < len ? qv[u] * qscale : 0.f;
      kl[s * LS + j] = s < len ? kv[u] : 0.f;
      sl[s * LS + j] = uv[u];
    }
    if (tid < 64) nl[tid] = d0 + tid < a.d ? un[d0 + tid] : 0.f;
    __syncthreads();
    for (int k = 0; k < 64; k += 4) {
      const float av = ql[(wave * 16 + lr) * LS + k + g];
#pragma unroll
      for (int j = 0; j < 4; j++) {
        sc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(
            av, kl[(j * 16 + lr) * LS + k + g], sc[j], 0, 0, 0);
        acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(
            av, sl[(k + g) * LS + j * 16 + lr], acc[j], 0, 0, 0);
      }
    }
#pragma unroll
    for (int j = 0; j < 16; j++)
      nq += ql[(tid >> 2) * LS + j * 4 + (tid & 3)] * nl[j * 4 + (tid & 3)];
  }
  nq += __shfl_xor(nq, 1);
  nq += __shfl_xor(nq, 2);
  __syncthreads();
  // values of the tile, and q.n per token
  {
    const int j = tid & 63;
    const bool vlive = vtile * VT + j < a.vd;
    const float* pv = a.P + a.ov + h * a.vd + vtile * VT + j;
    float vv[16];
#pragma unroll
    for (int u = 0; u < 16; u++)
      vv[u] = vlive
          ? pv[(size_t)(row0 + min(wave + u * 4, len - 1)) * a.ldp] : 0.f;
#pragma unroll
    for (int u = 0; u < 16; u++) {
      const int s = wave + u * 4;
      sl[s * LS + j] = s < len ? vv[u] : 0.f;
    }
  }
  if ((tid & 3) == 0) nl[tid >> 2] = nq;
  __syncthreads();
  float den[4];
#pragma unroll
  for (int r = 0; r < 4; r++) {
    const int t = wave * 16 + g * 4 + r;
    const float Ft = Fl[t], mt = ml[t];
    const float carry = expf(Ft + m0 - mt);
    float rs = 0.f;
#pragma unroll
    for (int j = 0; j < 4; j++) {
      const int s = j * 16 + lr;
      const float w = s <= t ? sc[j][r] * expf(Ft - Fl[s] + il[s] - mt) : 0.f;
      kl[t * LS + s] = w;                  // this wave's rows only
      rs += w;
      acc[j][r] *= carry;
    }
#pragma unroll
    for (int x = 1; x < 16; x <<= 1) rs += __shfl_xor(rs, x);
    den[r] = fmaxf(fabsf(carry * nl[t] + rs), expf(-mt)) + 1e-6f;
  }
  __syncthreads();
  for (int k = 0; k < CH; k += 4) {
    const float av = kl[(wave * 16 + lr) * LS + k + g];
#pragma unroll
    for (int j = 0; j < 4; j++)
      acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(
          av, sl[(k + g) * LS + j * 16 + lr], acc[j], 0, 0, 0);
  }
#pragma unroll
  for (int j = 0; j < 4; j++)
#pragma unroll
    for (int r = 0; r < 4; r++) {
      const int t = wave * 16 + g * 4 + r, v = vtile * VT + j * 16 + lr;
      if (t < len && v < a.vd)
        a.o[(size_t)(row0 + t) * a.H * a.vd + h * a.vd + v] =
            acc[j][r] / den[r];
    }
}

// per-head RMS norm, weight and sigmoid gate (one block per row); routes too
template <typename T>
__global__ void __launch_bounds__(256) k_mlstm_post(MlstmArgs a) {
  const int r = blockIdx.x, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const float* o = a.o + (size_t)r * a.H * a.vd;
  const float* gt = a.P + (size_t)r * a.ldp + a.og;
  T* out = (T*)a.out + (size_t)r * a.ldo;
  for (int h = wave; h < a.H; h += 4) {
    float ss = 0.f;
    for (int i = lane; i < a.vd; i += 64) {
      float v = o[h * a.vd + i];
      ss += v * v;
    }
    const float rn = 1.f / sqrtf(wave_reduce_sum(ss) / (float)a.vd + a.eps);
    for (int i = lane; i < a.vd; i += 64) {
      const int j = h * a.vd + i;
      out[j] = El<T>::st(o[j] * rn * a.norm[j] * sigmoid_f(gt[j]));
    }
  }
  if (a.E > 0 && wave == 0) {
    const float* z = a.P + (size_t)r * a.ldp + a.orouter;
    const int k1 = a.rtop + a.rextra;
    if (a.E <= 64)
      route_row<1>(z, a.E, a.rtop, a.rextra, a.ridx + r * k1, a.rwt + r * k1);
    else
      route_row<16>(z, a.E, a.rtop, a.rextra, a.ridx + r * k1, a.rwt + r * k1);
  }
}

// one block per (row, quarter of the heads) beside the experts' gate/up
template <typename T>
__global__ void __launch_bounds__(256) k_mlstm_dec_fin(MlstmArgs a, MoeArgs m,
                                                       int fblocks) {
  const int nmix = a.rows * ((a.H + 3) / 4);
  if ((int)blockIdx.x >= nmix) {
    const int b = blockIdx.x - nmix;
    expert_gu_block<T>(m, b / fblocks, b % fblocks);
    return;
  }
  const int hb = (a.H + 3) / 4;
  const int r = blockIdx.x / hb, lane = threadIdx.x & 63;
  const int h = (blockIdx.x - r * hb) * 4 + (threadIdx.x >> 6);
  if (h >= a.H) return;
  const float* o = a.o + (size_t)r * a.H * a.vd + h * a.vd;
  const float* gt = a.P + (size_t)r * a.ldp + a.og + h * a.vd;
  T* out = (T*)a.out + (size_t)r * a.ldo + h * a.vd;
  float ss = 0.f;
  for (int i = lane; i < a.vd; i += 64) ss += o[i] * o[i];
  const float rn = 1.f / sqrtf(wave_reduce_sum(ss) / (float)a.vd + a.eps);
  for (int i = lane; i < a.vd; i += 64)
    out[i] = El<T>::st(o[i] * rn * a.norm[h * a.vd + i] * sigmoid_f(gt[i]));
}

// ---- launchers ------------------------------------------------------------
static bool bad_shape(const MlstmArgs& a) {
  return a.rows < 1 || a.H < 1 || a.d < 1 || a.vd < 1 ||
         a.nvt != (a.vd + VT - 1) / VT || a.ldo < a.H * a.vd || a.E > 1024 ||
         (a.E > 0 && a.rtop > a.E) || a.d > 8192;
}

extern "C" hipError_t launch_mlstm_step(const MlstmArgs* a, hipStream_t s) {
  if (bad_shape(*a)) return hipErrorInvalidValue;
  size_t lds = (size_t)(2 * a->d + SW * VT) * sizeof(float);
  RAISE_LDS(k_mlstm_step);
  hipLaunchKernelGGL(k_mlstm_step,
                     dim3(a->H * a->nvt + (a->E > 0 ? 1 : 0), a->rows),
                     dim3(64 * SW), lds, s, *a);
  return hipGetLastError();
}

// gates, local sums, scan, outputs over the segments' rows
extern "C" hipError_t launch_mlstm_chunks(const MlstmArgs* a, hipStream_t s) {
  if (bad_shape(*a) || a->nseg < 1 || a->nchunk < 1)
    return hipErrorInvalidValue;
  const int ndt = (a->d + 63) / 64;
  hipLaunchKernelGGL(k_mlstm_gates, dim3(a->H, a->nchunk), dim3(64), 0, s, *a);
  hipLaunchKernelGGL(k_mlstm_chain, dim3(a->H, a->nseg), dim3(64), 0, s, *a);
  hipLaunchKernelGGL(k_mlstm_local, dim3(ndt * a->nvt, a->nchunk, a->H),
                     dim3(256), 0, s, *a);
  hipLaunchKernelGGL(k_mlstm_scan,
                     dim3((a->d * a->vd + a->d + 255) / 256, a->H, a->nseg),
                     dim3(256), 0, s, *a);
  size_t lds = (size_t)(3 * CH * LS + 4 * CH) * sizeof(float);
  RAISE_LDS(k_mlstm_out);
  hipLaunchKernelGGL(k_mlstm_out, dim3(a->nvt, a->nchunk, a->H), dim3(256),
                     lds, s, *a);
  return hipGetLastError();
}

extern "C" hipError_t launch_mlstm_post(int f32, const MlstmArgs* a,
                                        hipStream_t s) {
  if (bad_shape(*a)) return hipErrorInvalidValue;
  if (f32) hipLaunchKernelGGL(k_mlstm_post<float>, dim3(a->rows), dim3(256), 0, s, *a);
  else hipLaunchKernelGGL(k_mlstm_post<u16>, dim3(a->rows), dim3(256), 0, s, *a);
  return hipGetLastError();
}

extern "C" hipError_t launch_mlstm_dec_fin(int f32, const MlstmArgs* a,
                                           const MoeArgs* m, int pairs,
                                           hipStream_t s) {
  if (bad_shape(*a)) return hipErrorInvalidValue;
  int ffm = m->ff > m->ffs ? m->ff : m->ffs;
  int fb = pairs ? (ffm + MOE_FPB - 1) / MOE_FPB : 1;
  dim3 grid(a->rows * ((a->H + 3) / 4) + pairs * fb);
  if (f32) hipLaunchKernelGGL(k_mlstm_dec_fin<float>, grid, dim3(256), 0, s, *a, *m, fb);
  else hipLaunchKernelGGL(k_mlstm_dec_fin<u16>, grid, dim3(256), 0, s, *a, *m, fb);
  return hipGetLastError();
}
