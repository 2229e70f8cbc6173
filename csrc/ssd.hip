// ssd.hip — state-space recurrence (Mamba-2) behind a short convolution.
//
//   x, B, C = silu of a causal convolution per channel, with bias
//   dt = softplus(projection + dtb),  log a = rate[h] dt   (rate = -exp(A_log))
//   S_t = a S_{t-1} + dt B_t x_t^T,   y_t = S_t^T C_t + D[h] x_t
//   out = y_t silu(z_t)
//
// Head h uses B and C of group h / (H/G).  Everything is fp32; products run
// on fp32 MFMA (16x16x4) for both activation types.
//
// State, one slot per sequence: S [slot, H, N, vd], and a ring of the last
// `taps` inputs of the convolution [slot, taps, C], the input of position p
// at p % taps, so a step writes an entry that no block of it reads.
// Positions before 0 read as zero whatever the slot held.
//
// Runs of tokens use the chunkwise form over 64 tokens.  L is the running sum
// of log a inside a chunk: token s reaches token t with exp(L_t - L_s), the
// state before the chunk with exp(L_t).
#include "gemm_tile.h"
#include "hybrid.h"

#define CH 64     // chunk length
#define VT 64     // value columns of a tile
#define LS 68     // LDS row stride of a 64-wide fp32 tile

struct SsdArgs {
  const float* P;             // fp32 projections [rows, ldp]
  const float *cw, *cb;       // [taps, C], [C]
  const float *dtb, *rate, *D;   // [H]
  float *S, *ring;
  float* u;                   // [rows, C]: convolved x | B | C
  float *dt, *L;              // [rows, H]
  float* U;                   // [chunks, H, N, vd]
  float* o;                   // gated outputs [rows, H*vd]
  const int *slot, *pos;      // per row
  const int *seg_row0, *seg_len, *seg_slot, *seg_pos0, *seg_chunk0;
  const int *chunk_row0, *chunk_len, *chunk_seg;
  int ldp, oz, ox, odt, H, G, N, vd, C, taps, nvt, rows, nseg, nchunk;
};

DEVINL float softplus_f(float z) {
  return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z)));
}

// first channels of B and C of a head, among the convolved ones
DEVINL int b_channel(const SsdArgs& a, int h) {
  return a.H * a.vd + h / (a.H / a.G) * a.N;
}
DEVINL int c_channel(const SsdArgs& a, int h) {
  return b_channel(a, h) + a.G * a.N;
}

// ---- one token per row ------------------------------------------------
// SW waves per (head, column tile): a wave's lanes own the 64 columns, the
// rows of S are dealt to the waves.  The first 128 rows are on their way
// while the convolutions are worked out.
template <int SW>
__global__ void __launch_bounds__(64 * SW) k_ssd_step(SsdArgs a) {
  constexpr int SPRE = 128 / SW;
  extern __shared__ float sm[];           // B[N], C[N], part[SW*64]
  const int r = blockIdx.y;
  const int h = blockIdx.x / a.nvt, vtile = blockIdx.x - h * a.nvt;
  const int tid = threadIdx.x, c = tid & 63, w = tid >> 6;
  float *bs = sm, *cs = sm + a.N, *part = sm + 2 * a.N;
  const float* p = a.P + (size_t)r * a.ldp;
  const size_t slot = a.slot[r];
  const int pos = a.pos[r], now = pos % a.taps;
  const int col = vtile * VT + c;
  const bool live = col < a.vd, fresh = pos == 0;
  float* S = a.S + ((slot * a.H + h) * a.N) * a.vd + col;
  float pre[SPRE];
#pragma unroll
  for (int u = 0; u < SPRE; u++) {
    const int i = w + u * SW;
    pre[u] = (live && !fresh && i < a.N) ? S[(size_t)i * a.vd] : 0.f;
  }
  float* ring = a.ring + slot * a.taps * a.C;
  auto conv = [&](int ch) {
    float u = a.cb[ch];
    for (int j = a.taps - 1; j >= 1; j--)        // input j places back
      if (j <= pos)
        u = fmaf(a.cw[(a.taps - 1 - j) * a.C + ch],
                 ring[(now >= j ? now - j : now - j + a.taps) * a.C + ch], u);
    return fast_silu(fmaf(a.cw[(a.taps - 1) * a.C + ch], p[a.ox + ch], u));
  };
  const float v = live ? conv(h * a.vd + col) : 0.f;
  const float dt = softplus_f(p[a.odt + h] + a.dtb[h]);
  const float keep = fast_exp(a.rate[h] * dt);
  const int b0 = b_channel(a, h), c0 = c_channel(a, h);
  for (int i = tid; i < 2 * a.N; i += 64 * SW) {
    const bool second = i >= a.N;
    const float u = conv(second ? c0 + i - a.N : b0 + i);
    sm[i] = second ? u : u * dt;
  }
  __syncthreads();
  float acc = 0.f;
  if (live) {
#pragma unroll
    for (int u = 0; u < SPRE; u++) {
      const int i = w + u * SW;
      if (i < a.N) {
        const float s = fmaf(keep, pre[u], bs[i] * v);
        S[(size_t)i * a.vd] = s;
        acc = fmaf(s, cs[i], acc);
      }
    }
#pragma unroll 4
    for (int i = w + SPRE * SW; i < a.N; i += SW) {
      float s = bs[i] * v;
      if (!fresh) s = fmaf(keep, S[(size_t)i * a.vd], s);
      S[(size_t)i * a.vd] = s;
      acc = fmaf(s, cs[i], acc);
    }
  }
  part[w * VT + c] = acc;
  // nobody reads this entry of the ring
  float* to = ring + (size_t)now * a.C;
  if (w == 1 && live) to[h * a.vd + col] = p[a.ox + h * a.vd + col];
  if (vtile == 0 && h % (a.H / a.G) == 0)
    for (int i = tid; i < a.N; i += 64 * SW) {
      to[b0 + i] = p[a.ox + b0 + i];
      to[c0 + i] = p[a.ox + c0 + i];
    }
  __syncthreads();
  if (tid < VT && live) {
    float o = a.D[h] * v;
#pragma unroll
    for (int u = 0; u < SW; u++) o += part[u * VT + c];
    const int e = h * a.vd + col;
    a.o[(size_t)r * a.H * a.vd + e] = o * fast_silu(p[a.oz + e]);
  }
}

// ---- runs of tokens -----------------------------------------------------
// input of channel c at position p of a run (its first row0 holds pos0);
// p >= pos0 - taps + 1
DEVINL float run_input(const SsdArgs& a, const float* x, const float* ring,
                       int pos0, int p, int c) {
  if (p >= pos0) return x[(size_t)(p - pos0) * a.ldp + c];
  return p >= 0 ? ring[(size_t)(p % a.taps) * a.C + c] : 0.f;
}

// convolutions of a chunk, 64 channels a block, wave w tokens 16w .. 16w+15;
// further blocks: step sizes and L, a wave per head, a lane per token
#define HEADS_PER_BLOCK 4
__global__ void __launch_bounds__(256) k_ssd_conv(SsdArgs a, int cblocks) {
  const int lane = threadIdx.x & 63, wave = wave_index(), c = blockIdx.y;
  const int sg = a.chunk_seg[c], crow = a.chunk_row0[c], len = a.chunk_len[c];
  if ((int)blockIdx.x >= cblocks) {
    const int h = (blockIdx.x - cblocks) * HEADS_PER_BLOCK + wave;
    if (h >= a.H) return;
    const size_t row = crow + min(lane, len - 1);
    const float dt = softplus_f(a.P[row * a.ldp + a.odt + h] + a.dtb[h]);
    float l = a.rate[h] * dt;
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) {
      const float v = __shfl_up(l, d);
      if (lane >= d) l += v;
    }
    if (lane < len) {
      a.dt[row * a.H + h] = dt;
      a.L[row * a.H + h] = l;
    }
    return;
  }
  const int ch = blockIdx.x * 64 + lane;
  if (ch >= a.C) return;
  const int row0 = a.seg_row0[sg], pos0 = a.seg_pos0[sg];
  const float* x = a.P + (size_t)row0 * a.ldp + a.ox;
  const float* ring = a.ring + (size_t)a.seg_slot[sg] * a.taps * a.C;
  const int at = pos0 + crow - row0, p0 = at + wave * 16;   // of the wave
  float u[16];
  const float b = a.cb[ch];
#pragma unroll
  for (int t = 0; t < 16; t++) u[t] = b;
  if (a.taps <= 4) {
    float w[4], xv[19];
#pragma unroll
    for (int q = 0; q < 4; q++)
      w[q] = q < a.taps ? a.cw[(a.taps - 1 - q) * a.C + ch] : 0.f;
#pragma unroll
    for (int t = 0; t < 19; t++) xv[t] = 0.f;
    if (p0 - 3 >= pos0 && p0 + 15 < at + len) {      // all in the run
      const float* xp = x + (size_t)(p0 - 3 - pos0) * a.ldp + ch;
#pragma unroll
      for (int t = 0; t < 19; t++) xv[t] = xp[(size_t)t * a.ldp];
    } else {
#pragma unroll
      for (int t = 0; t < 19; t++) {
        const int p = p0 + t - 3;
        if (p - at < len && p >= pos0 - a.taps + 1)
          xv[t] = run_input(a, x, ring, pos0, p, ch);
      }
    }
#pragma unroll
    for (int t = 0; t < 16; t++)
#pragma unroll
      for (int q = 3; q >= 0; q--) u[t] = fmaf(w[q], xv[t + 3 - q], u[t]);
  } else {
    for (int q = a.taps - 1; q >= 0; q--) {
      const float w = a.cw[(size_t)(a.taps - 1 - q) * a.C + ch];
#pragma unroll
      for (int t = 0; t < 16; t++)
        if (p0 + t - at < len)
          u[t] = fmaf(w, run_input(a, x, ring, pos0, p0 + t - q, ch), u[t]);
    }
  }
#pragma unroll
  for (int t = 0; t < 16; t++)
    if (wave * 16 + t < len)
      a.u[(size_t)(crow + wave * 16 + t) * a.C + ch] = fast_silu(u[t]);
}

// what a chunk adds to the state: U = sum_s exp(L_end - L_s) dt_s B_s x_s^T
__global__ void __launch_bounds__(256) k_ssd_local(SsdArgs a) {
  __shared__ __attribute__((aligned(16))) float kl[CH * LS], vl[CH * LS];
  const int c = blockIdx.y, h = blockIdx.z;
  const int nnt = (a.N + 63) / 64;
  const int vtile = blockIdx.x / nnt, nt = blockIdx.x - vtile * nnt;
  const int row0 = a.chunk_row0[c], len = a.chunk_len[c];
  const int tid = threadIdx.x, wave = wave_index(), lane = tid & 63;
  const int j = lane;
  const bool nl = nt * 64 + j < a.N, vlive = vtile * VT + j < a.vd;
  const float* pk = a.u + b_channel(a, h) + nt * 64 + j;
  const float* pv = a.u + h * a.vd + vtile * VT + j;
  const float end = a.L[(size_t)(row0 + len - 1) * a.H + h];
  float kv[16], vv[16], wt[16];
#pragma unroll
  for (int u = 0; u < 16; u++) {
    const size_t row = row0 + min(wave + u * 4, len - 1);
    kv[u] = nl ? pk[row * a.C] : 0.f;
    vv[u] = vlive ? pv[row * a.C] : 0.f;
    wt[u] = fast_exp(end - a.L[row * a.H + h]) * a.dt[row * a.H + h];
  }
#pragma unroll
  for (int u = 0; u < 16; u++) {
    const int s = wave + u * 4;
    kl[s * LS + j] = s < len ? kv[u] * wt[u] : 0.f;
    vl[s * LS + j] = vv[u];
  }
  __syncthreads();
  const int lr = lane & 15, g = lane >> 4;
  f4v acc[4];
#pragma unroll
  for (int q = 0; q < 4; q++) acc[q] = {0.f, 0.f, 0.f, 0.f};
  for (int s = 0; s < CH; s += 4) {
    const float av = kl[(s + g) * LS + wave * 16 + lr];
#pragma unroll
    for (int q = 0; q < 4; q++)
      acc[q] = __builtin_amdgcn_mfma_f32_16x16x4f32(
          av, vl[(s + g) * LS + q * 16 + lr], acc[q], 0, 0, 0);
  }
  float* U = a.U + ((size_t)c * a.H + h) * a.N * a.vd;
#pragma unroll
  for (int q = 0; q < 4; q++)
#pragma unroll
    for (int r = 0; r < 4; r++) {
      const int ni = nt * 64 + wave * 16 + g * 4 + r;
      const int vi = vtile * VT + q * 16 + lr;
      if (ni < a.N && vi < a.vd) U[(size_t)ni * a.vd + vi] = acc[q][r];
    }
}

// carry the state over the chunks; U becomes the state BEFORE each chunk
__global__ void __launch_bounds__(256) k_ssd_scan(SsdArgs a) {
  const int h = blockIdx.y, sg = blockIdx.z;
  const int i = blockIdx.x * 256 + threadIdx.x;
  const int nv = a.N * a.vd;
  if (i >= nv) return;
  const int c0 = a.seg_chunk0[sg], nc = (a.seg_len[sg] + CH - 1) / CH;
  float* st = a.S + ((size_t)a.seg_slot[sg] * a.H + h) * nv + i;
  float cur = a.seg_pos0[sg] == 0 ? 0.f : *st;
  for (int c = c0; c < c0 + nc; c += 8) {
    const int n = min(8, c0 + nc - c);
    float* u = a.U + ((size_t)c * a.H + h) * nv + i;
    float add[8], dec[8];
#pragma unroll
    for (int k = 0; k < 8; k++) {
      add[k] = k < n ? u[(size_t)k * a.H * nv] : 0.f;
      const int cc = c + min(k, n - 1);
      dec[k] = a.L[(size_t)(a.chunk_row0[cc] + a.chunk_len[cc] - 1) * a.H + h];
    }
#pragma unroll
    for (int k = 0; k < 8; k++)
      if (k < n) {
        u[(size_t)k * a.H * nv] = cur;
        cur = fmaf(fast_exp(dec[k]), cur, add[k]);
      }
  }
  *st = cur;
}

// outputs of a chunk: wave w holds tokens 16w .. 16w+15
__global__ void __launch_bounds__(256) k_ssd_out(SsdArgs a) {
  __shared__ __attribute__((aligned(16))) float ql[CH * LS], kl[CH * LS],
      sl[CH * LS];
  __shared__ float Ls[CH], ds[CH];
  const int vtile = blockIdx.x, c = blockIdx.y, h = blockIdx.z;
  const int row0 = a.chunk_row0[c], len = a.chunk_len[c];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int lr = lane & 15, g = lane >> 4, j = lane;
  const float* U = a.U + ((size_t)c * a.H + h) * a.N * a.vd;
  const int v = vtile * VT + j;
  const bool vlive = v < a.vd;
  if (tid < CH) {
    const size_t row = row0 + min(tid, len - 1);
    Ls[tid] = a.L[row * a.H + h];
    ds[tid] = a.dt[row * a.H + h];
  }
  f4v sc[4], acc[4];
#pragma unroll
  for (int q = 0; q < 4; q++)
    sc[q] = acc[q] = f4v{0.f, 0.f, 0.f, 0.f};
  for (int n0 = 0; n0 < a.N; n0 += 64) {
    const bool nl = n0 + j < a.N;
    const float* pq = a.u + c_channel(a, h) + n0 + j;
    const float* pk = a.u + b_channel(a, h) + n0 + j;
    float qv[16], kv[16], uv[16];
#pragma unroll
    for (int u = 0; u < 16; u++) {
      const int s = wave + u * 4;            // a token, and a row of U
      const size_t row = row0 + min(s, len - 1);
      qv[u] = nl ? pq[row * a.C] : 0.f;
      kv[u] = nl ? pk[row * a.C] : 0.f;
      uv[u] = (n0 + s < a.N && vlive) ? U[(size_t)(n0 + s) * a.vd + v] : 0.f;
    }
    if (n0) __syncthreads();
#pragma unroll
    for (int u = 0; u < 16; u++) {
      const int s = wave + u * 4;
      ql[s * LS + j] = s < len ? qv[u] : 0.f;
      kl[s * LS + j] = s < len ? kv[u] : 0.f;
      sl[s * LS + j] = uv[u];
    }
    __syncthreads();
    for (int k = 0; k < 64; k += 16) {
      const f4v qf = ld16(ql + (wave * 16 + lr) * LS + k + g * 4);
#pragma unroll
      for (int q = 0; q < 4; q++) {
        sc[q] = GemmMma<float>::mma(
            qf, ld16(kl + (q * 16 + lr) * LS + k + g * 4), sc[q]);
#pragma unroll
        for (int i = 0; i < 4; i++)
          acc[q] = __builtin_amdgcn_mfma_f32_16x16x4f32(
              qf[i], sl[(k + g * 4 + i) * LS + q * 16 + lr], acc[q], 0, 0, 0);
      }
    }
  }
  __syncthreads();
  {
    const float* pv = a.u + h * a.vd + v;
    float vv[16];
#pragma unroll
    for (int u = 0; u < 16; u++)
      vv[u] = vlive ? pv[(size_t)(row0 + min(wave + u * 4, len - 1)) * a.C] : 0.f;
#pragma unroll
    for (int u = 0; u < 16; u++) {
      const int s = wave + u * 4;
      sl[s * LS + j] = s < len ? vv[u] : 0.f;
    }
  }
#pragma unroll
  for (int r = 0; r < 4; r++) {
    const int t = wave * 16 + g * 4 + r;
    const float lt = Ls[t], carry = fast_exp(lt);
#pragma unroll
    for (int q = 0; q < 4; q++) {
      const int s = q * 16 + lr;
      kl[t * LS + s] = s <= t ? sc[q][r] * fast_exp(lt - Ls[s]) * ds[s] : 0.f;
      acc[q][r] *= carry;
    }
  }
  __syncthreads();
  for (int k = 0; k < wave * 16 + 16; k += 16) {      // keys up to the wave's
    const f4v pf = ld16(kl + (wave * 16 + lr) * LS + k + g * 4);
#pragma unroll
    for (int q = 0; q < 4; q++)
#pragma unroll
      for (int i = 0; i < 4; i++)
        acc[q] = __builtin_amdgcn_mfma_f32_16x16x4f32(
            pf[i], sl[(k + g * 4 + i) * LS + q * 16 + lr], acc[q], 0, 0, 0);
  }
  const float skip = a.D[h];
#pragma unroll
  for (int q = 0; q < 4; q++)
#pragma unroll
    for (int r = 0; r < 4; r++) {
      const int t = wave * 16 + g * 4 + r, vi = vtile * VT + q * 16 + lr;
      if (t < len && vi < a.vd) {
        const size_t row = row0 + t;
        const int e = h * a.vd + vi;
        a.o[row * a.H * a.vd + e] =
            fmaf(skip, sl[t * LS + q * 16 + lr], acc[q][r]) *
            fast_silu(a.P[row * a.ldp + a.oz + e]);
      }
    }
  // the run's last inputs of the convolution
  const int sg = a.chunk_seg[c], seg0 = a.seg_row0[sg], slen = a.seg_len[sg];
  if (row0 + len != seg0 + slen) return;
  float* ring = a.ring + (size_t)a.seg_slot[sg] * a.taps * a.C;
  const bool shared = vtile == 0 && h % (a.H / a.G) == 0;
  for (int q = wave; q < min(a.taps, slen); q += 4) {
    const size_t row = seg0 + slen - 1 - q;
    const float* x = a.P + row * a.ldp + a.ox;
    float* to = ring + (size_t)((a.seg_pos0[sg] + slen - 1 - q) % a.taps) * a.C;
    if (vlive) to[h * a.vd + v] = x[h * a.vd + v];
    if (shared)
      for (int i = lane; i < a.N; i += 64) {
        const int b = b_channel(a, h) + i, cc = c_channel(a, h) + i;
        to[b] = x[b];
        to[cc] = x[cc];
      }
  }
}

// ---- launchers ------------------------------------------------------------
static bool bad_shape(const SsdArgs& a) {
  return a.rows < 1 || a.H < 1 || a.G < 1 || a.H % a.G || a.N < 1 ||
         a.N > 8192 || a.vd < 1 || a.nvt != (a.vd + VT - 1) / VT ||
         a.C != a.H * a.vd + 2 * a.G * a.N || a.taps < 1;
}

template <int SW> static hipError_t step_go(const SsdArgs& a, hipStream_t s) {
  const size_t lds = (size_t)(2 * a.N + SW * VT) * sizeof(float);
  RAISE_LDS(k_ssd_step<SW>);
  hipLaunchKernelGGL(k_ssd_step<SW>, dim3(a.H * a.nvt, a.rows), dim3(64 * SW),
                     lds, s, a);
  return hipGetLastError();
}

extern "C" hipError_t launch_ssd_step(const SsdArgs* a, hipStream_t s) {
  if (bad_shape(*a)) return hipErrorInvalidValue;
  // two blocks of 16 waves fill a CU; beyond that more, smaller ones
  return a->H * a->nvt * a->rows <= 512 ? step_go<16>(*a, s)
                                        : step_go<4>(*a, s);
}

// convolutions, local sums, scan, outputs over the segments' rows
extern "C" hipError_t launch_ssd_run(const SsdArgs* a, hipStream_t s) {
  if (bad_shape(*a) || a->nseg < 1 || a->nchunk < 1)
    return hipErrorInvalidValue;
  const int cb = (a->C + 63) / 64, nnt = (a->N + 63) / 64;
  const int hb = (a->H + HEADS_PER_BLOCK - 1) / HEADS_PER_BLOCK;
  hipLaunchKernelGGL(k_ssd_conv, dim3(cb + hb, a->nchunk), dim3(256), 0, s, *a,
                     cb);
  hipLaunchKernelGGL(k_ssd_local, dim3(nnt * a->nvt, a->nchunk, a->H),
                     dim3(256), 0, s, *a);
  hipLaunchKernelGGL(k_ssd_scan, dim3((a->N * a->vd + 255) / 256, a->H, a->nseg),
                     dim3(256), 0, s, *a);
  hipLaunchKernelGGL(k_ssd_out, dim3(a->nvt, a->nchunk, a->H), dim3(256), 0, s,
                     *a);
  return hipGetLastError();
}
