// linear.hip — embedding, norm and linear kernels around an fp32 residual
// stream.  Weights are T = bf16 or float, stored [N, Kp] with the K axis
// zero-padded to a multiple of 64; projections come out in fp32.
#include <type_traits>

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

// ---- embedding of tokens and token pairs ---------------------------------
// x = table[cur] + pairs[(before * mul_before + cur * mul_cur) mod buckets],
// the last row of pairs at position 0, once for each of S streams.  The token
// before a sequence's next one is kept in last[slot]; the runs' last tokens
// are written by a launch of their own, since their first rows read the entry.
struct PairEmbed {
  const void *table, *pairs;   // [vocab, W], [buckets + 1, W]
  const int *ids, *slot, *pos;
  int* last;                   // [slots]
  float* x;                    // [rows, S, W]
  const int *seg_row0, *seg_len, *seg_slot;   // runs
  long mul_before, mul_cur;
  int W, S, M, nd, nseg, buckets;   // rows [0, nd) are single tokens
};

template <typename T>
__global__ void __launch_bounds__(256) k_embed_pairs(PairEmbed a) {
  const int r = blockIdx.x, W = a.W, cur = a.ids[r], slot = a.slot[r];
  long row = a.buckets;
  if (a.pos[r] > 0) {
    const bool inside = r > 0 && a.slot[r - 1] == slot;   // of a run
    const long before = inside ? a.ids[r - 1] : a.last[slot];
    row = (before * a.mul_before + cur * a.mul_cur) % a.buckets;
  }
  if (r < a.nd) {
    __syncthreads();                     // everyone has the entry
    if (threadIdx.x == 0) a.last[slot] = cur;
  }
  const T* t = (const T*)a.table + (size_t)cur * W;
  const T* p = (const T*)a.pairs + (size_t)row * W;
  for (int i = threadIdx.x; i < W; i += 256) {
    const float v = El<T>::ld(t[i]) + El<T>::ld(p[i]);
    for (int q = 0; q < a.S; q++) a.x[((size_t)r * a.S + q) * W + i] = v;
  }
}

__global__ void __launch_bounds__(256) k_last_tokens(PairEmbed a) {
  const int g = blockIdx.x * 256 + threadIdx.x;
  if (g < a.nseg)
    a.last[a.seg_slot[g]] = a.ids[a.seg_row0[g] + a.seg_len[g] - 1];
}

// ---- staging a row of the residual for a projection --------------------
// v = x [+ y / rms(y) * gb] [+ xadd]            (y: the last sublayer's output)
// out = v / rms(v) * g [* sigmoid(gate)]
// or, with CONV, v + a causal convolution over time on each channel,
//   out = v + sum_j cw[taps-1-j] v(pos - j),    zero before position 0.
// The last inputs v of a sequence are kept in a ring, ring[slot][pos % taps].
// A row of up to NT*U elements stays in the registers of NT threads.
struct RowStage {
  const float* x;
  const float *y, *gb;      // nullable pair
  const float* xadd;        // nullable
  const float* g;           // null: only v is wanted
  const float* gate;        // nullable, [rows, ldg]
  float* xout;              // nullable: receives v
  const float* cw;          // CONV: [taps, W]
  float* ring;              // CONV: [slots, taps, W]
  const int *slot, *pos;    // CONV: per row
  int W, Kp, ldg, taps;
  float eps;
};

template <int NT, int U, bool CONV = false, class Put>
DEVINL void stage_row(const RowStage& s, size_t row, bool keep, float* red,
                      Put put) {
  const int tid = threadIdx.x, W = s.W;
  const size_t o = row * W;
  float xv[U], gv[U], yv[U];
#pragma unroll
  for (int u = 0; u < U; u++) {
    const int i = tid + u * NT;
    xv[u] = i < W ? s.x[o + i] : 0.f;
    gv[u] = s.g && i < W ? s.g[i] : 0.f;
    if (s.y) yv[u] = i < W ? s.y[o + i] : 0.f;
  }
  [[maybe_unused]] int pos = 0;
  [[maybe_unused]] float* ring = nullptr;
  [[maybe_unused]] float cv[U], cl[U];   // earlier inputs' part, newest tap
  if constexpr (CONV) {
    pos = s.pos[row];
    ring = s.ring + (size_t)s.slot[row] * s.taps * W;
    const int now = pos % s.taps;
    // input j places back; the first three without branches, so that their
    // loads are on the way together
    float h[3][U], c[3][U];
#pragma unroll
    for (int j = 1; j <= 3; j++) {
      const bool ok = j < s.taps && j <= pos;
      const float* hp = ring + (ok ? now - j + (now < j ? s.taps : 0) : 0) * W;
      const float* cp = s.cw + (ok ? s.taps - 1 - j : 0) * W;
#pragma unroll
      for (int u = 0; u < U; u++) {
        const int i = min(tid + u * NT, W - 1);
        h[j - 1][u] = hp[i];
        c[j - 1][u] = cp[i];
        if (!ok) h[j - 1][u] = c[j - 1][u] = 0.f;     // may hold anything
      }
    }
#pragma unroll
    for (int u = 0; u < U; u++) {
      const int i = tid + u * NT;
      cl[u] = i < W ? s.cw[(size_t)(s.taps - 1) * W + i] : 0.f;
      cv[u] = 0.f;
#pragma unroll
      for (int j = 0; j < 3; j++) cv[u] = fmaf(c[j][u], h[j][u], cv[u]);
    }
    for (int j = 4; j < s.taps && j <= pos; j++) {
      const float* hp = ring + (size_t)((pos - j) % s.taps) * W;
      const float* cp = s.cw + (size_t)(s.taps - 1 - j) * W;
#pragma unroll
      for (int u = 0; u < U; u++) {
        const int i = tid + u * NT;
        if (i < W) cv[u] = fmaf(cp[i], hp[i], cv[u]);
      }
    }
  }
  float rb = 0.f;
  if (s.y) {
    float ss = 0.f, gb[U];
#pragma unroll
    for (int u = 0; u < U; u++) {
      const int i = tid + u * NT;
      gb[u] = i < W ? s.gb[i] : 0.f;
      ss += yv[u] * yv[u];
    }
    for (int i = tid + U * NT; i < W; i += NT) ss += s.y[o + i] * s.y[o + i];
    rb = 1.f / sqrtf(block_sum(ss, red) / (float)W + s.eps);
#pragma unroll
    for (int u = 0; u < U; u++) xv[u] += yv[u] * rb * gb[u];
  }
  if (s.xadd)
#pragma unroll
    for (int u = 0; u < U; u++) {
      const int i = tid + u * NT;
      if (i < W) xv[u] += s.xadd[o + i];
    }
  auto late = [&](int i) {              // elements beyond the registers
    float v = s.x[o + i];
    if (s.y) v += s.y[o + i] * rb * s.gb[i];
    if (s.xadd) v += s.xadd[o + i];
    return v;
  };
  float rn = 0.f;
  if (s.g) {
    float ss = 0.f;
#pragma unroll
    for (int u = 0; u < U; u++) ss += xv[u] * xv[u];
    for (int i = tid + U * NT; i < W; i += NT) {
      const float v = late(i);
      ss += v * v;
    }
    rn = 1.f / sqrtf(block_sum(ss, red) / (float)W + s.eps);
  }
  const float* gt = s.gate ? s.gate + row * s.ldg : nullptr;
  auto finish = [&](int i, float v, float g) {
    if (s.g && i < s.Kp)
      put(i, i < W ? v * rn * g * (gt ? sigmoid_f(gt[i]) : 1.f) : 0.f);
    // xout may be x: its reads are done
    if (keep && s.xout && i < W) s.xout[o + i] = v;
  };
  if constexpr (CONV) {
    auto mix = [&](int i, float v, float c, float before) {
      if (i < s.Kp) put(i, i < W ? v + fmaf(c, v, before) : 0.f);
      if (keep && i < W) {
        if (s.xout) s.xout[o + i] = v;
        ring[(size_t)(pos % s.taps) * W + i] = v;   // nobody reads this entry
      }
    };
#pragma unroll
    for (int u = 0; u < U; u++) mix(tid + u * NT, xv[u], cl[u], cv[u]);
    for (int i = tid + U * NT; i < max(W, s.Kp); i += NT) {
      float before = 0.f;
      if (i < W)
        for (int j = 1; j < s.taps && j <= pos; j++)
          before = fmaf(s.cw[(size_t)(s.taps - 1 - j) * W + i],
                        ring[(size_t)((pos - j) % s.taps) * W + i], before);
      mix(i, i < W ? late(i) : 0.f,
          i < W ? s.cw[(size_t)(s.taps - 1) * W + i] : 0.f, before);
    }
    return;
  }
#pragma unroll
  for (int u = 0; u < U; u++) finish(tid + u * NT, xv[u], gv[u]);
  for (int i = tid + U * NT; i < max(W, s.Kp); i += NT)
    finish(i, i < W ? late(i) : 0.f, s.g && i < W ? s.g[i] : 0.f);
}

// ---- staging a row of several residual streams ----------------------------
// With the output y of the sublayer before (or two halves of it,
// y = (y / rms(y) gb + y2 / rms(y2) gb2) / 2), all streams at once:
//   x_t <- sum_s mix[s][t] x_s + feed[t] y
// then u = sum_s in[s] x_s and out = u / rms(u) * g, g a single number.
#define MAX_STREAMS 8
struct HyperStage {
  const float* x;           // [rows, S, W]
  const float *y, *y2;      // nullable, [rows, W]
  const float *gb, *gb2;    // with y2
  const float *mix, *feed;  // with y: [S, S], [S]
  const float *in, *g;      // [S], [1]; null: only xout is wanted
  float* xout;              // nullable: receives the streams
  int W, Kp, S;
  float eps;
};

// HS streams, or s.S of them where HS is 0
template <int NT, int U, int HS, class Put>
DEVINL void stage_hyper(const HyperStage& s, size_t row, bool keep, float* red,
                        Put put) {
  constexpr int MS = HS ? HS : MAX_STREAMS;
  const int tid = threadIdx.x, W = s.W, S = HS ? HS : s.S;
  const float* x = s.x + row * S * W;
  const float* y = s.y ? s.y + row * W : nullptr;
  const float* y2 = s.y2 ? s.y2 + row * W : nullptr;
  float xv[U][MS], yv[U], zv[U], ga[U], gc[U];
#pragma unroll
  for (int u = 0; u < U; u++) {
    const int i = tid + u * NT;
#pragma unroll
    for (int t = 0; t < MS; t++)
      xv[u][t] = t < S && i < W ? x[(size_t)t * W + i] : 0.f;
    yv[u] = y && i < W ? y[i] : 0.f;
    zv[u] = y2 && i < W ? y2[i] : 0.f;
    ga[u] = y2 && i < W ? s.gb[i] : 0.f;
    gc[u] = y2 && i < W ? s.gb2[i] : 0.f;
  }
  float ra = 1.f, rc = 0.f;
  if (y2) {
    float sa = 0.f, sc = 0.f;
#pragma unroll
    for (int u = 0; u < U; u++) {
      sa += yv[u] * yv[u];
      sc += zv[u] * zv[u];
    }
    for (int i = tid + U * NT; i < W; i += NT) {
      sa += y[i] * y[i];
      sc += y2[i] * y2[i];
    }
    ra = 0.5f / sqrtf(block_sum(sa, red) / (float)W + s.eps);
    rc = 0.5f / sqrtf(block_sum(sc, red) / (float)W + s.eps);
  }
  // the streams of one element, and what the next sublayer reads of them
  auto turn = [&](float (&v)[MS], float yo) {
    if (y) {
      float n[MS];
#pragma unroll
      for (int t = 0; t < MS; t++) {
        n[t] = 0.f;
        if (t < S) {
          n[t] = s.feed[t] * yo;
#pragma unroll
          for (int q = 0; q < MS; q++)
            if (q < S) n[t] = fmaf(s.mix[q * S + t], v[q], n[t]);
        }
      }
#pragma unroll
      for (int t = 0; t < MS; t++) v[t] = n[t];
    }
    float u = 0.f;
    if (s.in)
#pragma unroll
      for (int t = 0; t < MS; t++)
        if (t < S) u = fmaf(s.in[t], v[t], u);
    return u;
  };
  auto late = [&](int i, float (&v)[MS]) {   // elements beyond the registers
#pragma unroll
    for (int t = 0; t < MS; t++) v[t] = t < S ? x[(size_t)t * W + i] : 0.f;
    float yo = y ? y[i] : 0.f;
    if (y2) yo = yo * ra * s.gb[i] + y2[i] * rc * s.gb2[i];
    return turn(v, yo);
  };
  float uv[U], ss = 0.f;
#pragma unroll
  for (int u = 0; u < U; u++) {
    const float yo = y2 ? yv[u] * ra * ga[u] + zv[u] * rc * gc[u] : yv[u];
    uv[u] = turn(xv[u], yo);
    ss += uv[u] * uv[u];
  }
  float rn = 0.f;
  if (s.in) {
    for (int i = tid + U * NT; i < W; i += NT) {
      float v[MS];
      const float u = late(i, v);
      ss += u * u;
    }
    rn = s.g[0] / sqrtf(block_sum(ss, red) / (float)W + s.eps);
  }
  auto finish = [&](int i, float u, const float (&v)[MS]) {
    if (s.in && i < s.Kp) put(i, i < W ? u * rn : 0.f);
    if (keep && s.xout && i < W)         // may be x: its reads are done
#pragma unroll
      for (int t = 0; t < MS; t++)
        if (t < S) s.xout[(row * S + t) * W + i] = v[t];
  };
#pragma unroll
  for (int u = 0; u < U; u++) finish(tid + u * NT, uv[u], xv[u]);
  for (int i = tid + U * NT; i < max(W, s.Kp); i += NT) {
    float v[MS];
    const float u = i < W ? late(i, v) : 0.f;
    finish(i, u, v);
  }
}

template <typename T, int U, int HS>
__global__ void __launch_bounds__(256)
k_hyper_rows(HyperStage s, const int* __restrict__ rows, T* __restrict__ out) {
  __shared__ float red[4];
  T* o = out + (size_t)blockIdx.x * s.Kp;
  stage_hyper<256, U, HS>(s, rows ? rows[blockIdx.x] : blockIdx.x, true, red,
                          [&](int i, float v) { o[i] = El<T>::st(v); });
}

// ---- staging a row normed in equal parts -----------------------------------
// out = x / rms(x over its part) * g; rn holds MAX_GROUPS floats
#define MAX_GROUPS 1024
template <int NT, class Put>
DEVINL void stage_groups(const RowStage& s, int groups, size_t row, float* rn,
                         Put put) {
  constexpr int NW = NT / 64;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, W = s.W;
  const int gw = W / groups, parts = max(1, NW / groups);
  const float* x = s.x + row * W;
  for (int k = wave; k < groups * parts; k += NW) {
    const int grp = k / parts, p = k - grp * parts;
    float ss = 0.f;
#pragma unroll 4
    for (int i = p * 64 + lane; i < gw; i += parts * 64)
      ss += x[grp * gw + i] * x[grp * gw + i];
    ss = wave_reduce_sum(ss);
    if (lane == 0) rn[k] = ss;
  }
  __syncthreads();
#pragma unroll 4
  for (int i = tid; i < s.Kp; i += NT) {
    float v = 0.f;
    if (i < W) {
      float ss = 0.f;
      const int grp = i / gw;
      for (int p = 0; p < parts; p++) ss += rn[grp * parts + p];
      v = x[i] / sqrtf(ss / (float)gw + s.eps) * s.g[i];
    }
    put(i, v);
  }
}

template <typename T>
__global__ void __launch_bounds__(256)
k_group_rows(RowStage s, int groups, T* __restrict__ out) {
  __shared__ float rn[MAX_GROUPS];
  T* o = out + (size_t)blockIdx.x * s.Kp;
  stage_groups<256>(s, groups, blockIdx.x, rn,
                    [&](int i, float v) { o[i] = El<T>::st(v); });
}

// one block per row; `rows` (nullable) picks the source row of each output
// row.  out rows have Kp elements; the padding is written as zero.
template <typename T, int U>
__global__ void __launch_bounds__(256)
k_norm_rows(RowStage s, const int* __restrict__ rows, T* __restrict__ out) {
  __shared__ float red[4];
  T* o = out + (size_t)blockIdx.x * s.Kp;
  stage_row<256, U>(s, rows ? rows[blockIdx.x] : blockIdx.x, true, red,
               [&](int i, float v) { o[i] = El<T>::st(v); });
}

// ---- rows with their input convolution -----------------------------------
// out[r] = v_r + conv(v)_r with v = x [+ y / rms(y) * gb], for single tokens
// and runs of tokens.  A block takes one single token, or R rows of a chunk
// of a run; it computes the rows ahead of its own again.  The block at the
// head of a run reads the ring and, channel by channel in the same thread,
// leaves the run's last inputs in it.
#define CHUNK 64

struct ConvRows {
  RowStage s;               // x, y, gb, xout (beside x), cw, ring, slot, pos
  void* out;                // [rows, Kp] T
  const int *seg_row0, *seg_len, *seg_slot, *seg_pos0;   // runs
  const int *chunk_row0, *chunk_len, *chunk_seg;
  int nd, nseg, nchunk;     // rows [0, nd) are single tokens
};

struct ConvBlock {
  int row0, n, seg0, len, slot, pos0;   // rows of the block, its sequence's run
};

template <int R> DEVINL ConvBlock conv_block(const ConvRows& a) {
  int b = blockIdx.x;
  if (b < a.nd) return {b, 1, b, 1, a.s.slot[b], a.s.pos[b]};
  b -= a.nd;                // neighbours on one XCD: they share rows in its L2
  b = b % 8 * (a.nchunk * (CHUNK / R) / 8) + b / 8;
  const int c = b / (CHUNK / R), at = b % (CHUNK / R) * R;
  const int g = a.chunk_seg[c];
  return {a.chunk_row0[c] + at, min(R, a.chunk_len[c] - at), a.seg_row0[g],
          a.seg_len[g], a.seg_slot[g], a.seg_pos0[g]};
}

// sums over the wave of N values a lane, N a power of two: lane l < N gets
// the sum of value sum_slot<N>(l)
template <int N> DEVINL float wave_sums(float (&v)[N]) {
  const int lane = threadIdx.x & 63;
  int mask = 1;
#pragma unroll
  for (int half = N / 2; half >= 1; half /= 2, mask *= 2) {
    const bool up = lane & mask;
#pragma unroll
    for (int i = 0; i < half; i++) {
      const float keep = up ? v[i + half] : v[i];
      const float give = up ? v[i] : v[i + half];
      v[i] = keep + __shfl_xor(give, mask);
    }
  }
  float t = v[0];
#pragma unroll
  for (int m = N; m < 64; m *= 2) t += __shfl_xor(t, m);
  return t;
}
template <int N> DEVINL int sum_slot(int lane) {
  return N == 1 ? 0 : (int)(__brev((unsigned)lane) >> (32 - __builtin_ctz(N)));
}

DEVINL f4v mix4(f4v x, f4v y, f4v gb, float rn) {
  f4v v;
#pragma unroll
  for (int c = 0; c < 4; c++) v[c] = x[c] + y[c] * rn * gb[c];
  return v;
}

template <typename T> DEVINL void st4(T* p, f4v v) {
  if constexpr (sizeof(T) == 2) {
    union { T t[4]; uint64_t u; } o;
#pragma unroll
    for (int c = 0; c < 4; c++) o.t[c] = El<T>::st(v[c]);
    *(uint64_t*)p = o.u;
  } else *(f4v*)p = v;
}

// a thread owns four channels: 4 NT >= W, W % 4 == 0, TAPS - 1 <= R; R = 1
// where the batch has single tokens only
template <typename T, int TAPS, int NT, int R>
__global__ void __launch_bounds__(NT) k_conv_rows(ConvRows a) {
  constexpr int B = TAPS - 1, NW = NT / 64;
  constexpr int N = R == 1 ? 1 : R + B <= 8 ? 8 : 16;
  constexpr int E0 = R == 1 ? B : 0;    // first row whose norm may be needed
  static_assert(R + B <= 16 && (B <= R || R == 1));
  __shared__ float red[NW][N];
  const RowStage& s = a.s;
  const ConvBlock k = R == 1 ? ConvBlock{(int)blockIdx.x, 1, (int)blockIdx.x, 1,
                                         s.slot[blockIdx.x], s.pos[blockIdx.x]}
                             : conv_block<R>(a);
  if (k.n <= 0) return;
  const int W = s.W, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int c0 = tid * 4;
  const bool mine = c0 < W;
  const f4v zero = {0.f, 0.f, 0.f, 0.f};
  float* ring = s.ring + (size_t)k.slot * TAPS * W + c0;
  // 1 / rms of the rows whose squares' sums each thread has in ss
  auto rms_all = [&](float (&ss)[N]) {
    const float t = wave_sums<N>(ss);
    if (lane < N) red[wave][sum_slot<N>(lane)] = t;
    __syncthreads();
    if (tid < N) {
      float sum = 0.f;
#pragma unroll
      for (int w = 0; w < NW; w++) sum += red[w][tid];
      red[0][tid] = 1.f / sqrtf(sum / (float)W + s.eps);
    }
    __syncthreads();
  };
  auto square = [](f4v v) {
    return v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
  };

  f4v v[R + B], y[R + B], w[TAPS], gb = zero;
  float ss[N];
#pragma unroll
  for (int e = 0; e < N; e++) ss[e] = 0.f;
#pragma unroll
  for (int e = 0; e < R + B; e++) {
    v[e] = y[e] = zero;
    const int row = k.row0 - B + e, back = row - k.seg0;   // < 0: before it
    if (!mine || e - B >= k.n) continue;
    if (back >= 0) {
      v[e] = *(const f4v*)(s.x + (size_t)row * W + c0);
      if (s.y) y[e] = *(const f4v*)(s.y + (size_t)row * W + c0);
    } else if (k.pos0 + back >= 0) {
      v[e] = *(const f4v*)(ring + (size_t)((k.pos0 + back) % TAPS) * W);
    }
  }
#pragma unroll
  for (int j = 0; j < TAPS; j++)
    w[j] = mine ? *(const f4v*)(s.cw + (size_t)j * W + c0) : zero;
  if (s.y) {
    if (mine) gb = *(const f4v*)(s.gb + c0);
#pragma unroll
    for (int e = E0; e < R + B; e++) ss[e - E0] = square(y[e]);
    rms_all(ss);
#pragma unroll
    for (int e = E0; e < R + B; e++)
      v[e] = mix4(v[e], y[e], gb, red[0][e - E0]);
  }
#pragma unroll
  for (int e = 0; e < R; e++) {
    if (e >= k.n) break;
    f4v o = v[B + e];
#pragma unroll
    for (int c = 0; c < 4; c++) {
      float sum = 0.f;
#pragma unroll
      for (int j = 0; j < TAPS; j++) sum = fmaf(w[j][c], v[e + j][c], sum);
      o[c] += sum;
    }
    if (c0 < s.Kp)
      st4((T*)a.out + (size_t)(k.row0 + e) * s.Kp + c0, mine ? o : zero);
    if (mine && s.xout)
      *(f4v*)(s.xout + (size_t)(k.row0 + e) * W + c0) = v[B + e];
  }
  if (k.row0 != k.seg0 || B == 0) return;
  if (R == 1 || k.len == 1) {
    if (mine) *(f4v*)(ring + (size_t)(k.pos0 % TAPS) * W) = v[B];
  } else if constexpr (R > 1) {         // the run's last inputs
    f4v xt[TAPS], yt[TAPS];
#pragma unroll
    for (int e = 0; e < N; e++) ss[e] = 0.f;
#pragma unroll
    for (int e = 0; e < B; e++) {
      const int row = k.seg0 + k.len - B + e;
      const bool in = mine && row >= k.seg0;
      xt[e] = in ? *(const f4v*)(s.x + (size_t)row * W + c0) : zero;
      yt[e] = in && s.y ? *(const f4v*)(s.y + (size_t)row * W + c0) : zero;
      ss[e] = square(yt[e]);
    }
    if (s.y) {
      __syncthreads();                  // red[0] has been read
      rms_all(ss);
    }
#pragma unroll
    for (int e = 0; e < B; e++) {
      const int at = k.len - B + e;
      if (mine && at >= 0)
        *(f4v*)(ring + (size_t)((k.pos0 + at) % TAPS) * W) =
            s.y ? mix4(xt[e], yt[e], gb, red[0][e]) : xt[e];
    }
  }
}

// 1 / rms of one row of y, by one wave
DEVINL float wave_rms(const RowStage& s, int row) {
  const float* y = s.y + (size_t)row * s.W;
  float ss = 0.f;
#pragma unroll 8
  for (int i = threadIdx.x & 63; i < s.W; i += 64) ss += y[i] * y[i];
  return 1.f / sqrtf(wave_reduce_sum(ss) / (float)s.W + s.eps);
}

// any number of taps and any width; the ring is written by a launch of its own
#define ANY_R 8
template <typename T>
__global__ void __launch_bounds__(256) k_conv_rows_any(ConvRows a) {
  extern __shared__ float rnx[];        // ANY_R + taps - 1
  const RowStage& s = a.s;
  const ConvBlock k = conv_block<ANY_R>(a);
  if (k.n <= 0) return;
  const int W = s.W, B = s.taps - 1, tid = threadIdx.x;
  if (s.y)
    for (int e = tid >> 6; e < k.n + B; e += 4) {
      const int row = k.row0 - B + e;
      if (row < k.seg0) continue;
      const float r = wave_rms(s, row);
      if ((tid & 63) == 0) rnx[e] = r;
    }
  __syncthreads();
  const float* ring = s.ring + (size_t)k.slot * s.taps * W;
  for (int i = tid; i < s.Kp; i += 256)
    for (int e = 0; e < k.n; e++) {
      T* o = (T*)a.out + (size_t)(k.row0 + e) * s.Kp + i;
      if (i >= W) {
        *o = El<T>::st(0.f);
        continue;
      }
      float sum = 0.f, v = 0.f;
      for (int j = 0; j < s.taps; j++) {
        const int row = k.row0 + e - B + j, back = row - k.seg0;
        v = 0.f;
        if (back >= 0) {
          v = s.x[(size_t)row * W + i];
          if (s.y) v += s.y[(size_t)row * W + i] * rnx[e + j] * s.gb[i];
        } else if (k.pos0 + back >= 0) {
          v = ring[(size_t)((k.pos0 + back) % s.taps) * W + i];
        }
        sum = fmaf(s.cw[(size_t)j * W + i], v, sum);
      }
      *o = El<T>::st(v + sum);
      if (s.xout) s.xout[(size_t)(k.row0 + e) * W + i] = v;
    }
}

// last inputs of every sequence of the batch -> its ring; v holds the rows
__global__ void __launch_bounds__(256)
k_conv_ring(ConvRows a, const float* __restrict__ v) {
  const int b = blockIdx.x, W = a.s.W, taps = a.s.taps, g = b - a.nd;
  const bool one = b < a.nd;
  const int row0 = one ? b : a.seg_row0[g], len = one ? 1 : a.seg_len[g];
  const int slot = one ? a.s.slot[b] : a.seg_slot[g];
  const int pos0 = one ? a.s.pos[b] : a.seg_pos0[g];
  float* ring = a.s.ring + (size_t)slot * taps * W;
  for (int t = max(0, len - taps + 1); t < len; t++)
    for (int i = threadIdx.x; i < W; i += 256)
      ring[(size_t)((pos0 + t) % taps) * W + i] = v[(size_t)(row0 + t) * W + i];
}

// ---- polynomial activation of whole rows ---------------------------------
// out = c0 N(z) + c1 N(z^2) + c2 N(z^3) + c3, N dividing by the root mean
// square over the row's W values; zero from W to Kp.
struct PolyNorm {
  float r1, r2, r3, e;
  DEVINL float operator()(float z) const {
    const float z2 = z * z;
    return r1 * z + (r2 * z2 + (r3 * (z2 * z) + e));
  }
};

// NT threads hold z[u] = element tid + u*NT, late(i) reads the others
template <int NT, int U, class Late>
DEVINL PolyNorm poly_moments(const float (&z)[U], Late late, int W,
                             const float* coef, float eps, float* red) {
  float m[3] = {0.f, 0.f, 0.f};
  auto add = [&](float v) {
    const float v2 = v * v, v4 = v2 * v2;
    m[0] += v2; m[1] += v4; m[2] += v4 * v2;
  };
#pragma unroll
  for (int u = 0; u < U; u++) add(z[u]);
  for (int i = threadIdx.x + U * NT; i < W; i += NT) add(late(i));
#pragma unroll
  for (int k = 0; k < 3; k++) m[k] = wave_reduce_sum(m[k]);
  if ((threadIdx.x & 63) == 0)
#pragma unroll
    for (int k = 0; k < 3; k++) red[(threadIdx.x >> 6) * 3 + k] = m[k];
  __syncthreads();
  float r[3];
#pragma unroll
  for (int k = 0; k < 3; k++) {
    float t = 0.f;
    for (int w = 0; w < NT / 64; w++) t += red[w * 3 + k];
    r[k] = coef[k] / sqrtf(t / (float)W + eps);
  }
  return {r[0], r[1], r[2], coef[3]};
}

template <typename T, int U>
__global__ void __launch_bounds__(256)
k_poly_rows(const float* __restrict__ z, int ldz, const float* __restrict__ coef,
            T* __restrict__ out, int W, int Kp, float eps) {
  __shared__ float red[12];
  const float* zr = z + (size_t)blockIdx.x * ldz;
  T* o = out + (size_t)blockIdx.x * Kp;
  float v[U];
#pragma unroll
  for (int u = 0; u < U; u++) {
    const int i = threadIdx.x + u * 256;
    v[u] = i < W ? zr[i] : 0.f;
  }
  auto late = [&](int i) { return zr[i]; };
  const PolyNorm f = poly_moments<256, U>(v, late, W, coef, eps, red);
#pragma unroll
  for (int u = 0; u < U; u++) {
    const int i = threadIdx.x + u * 256;
    if (i < Kp) o[i] = El<T>::st(i < W ? f(v[u]) : 0.f);
  }
  for (int i = threadIdx.x + U * 256; i < Kp; i += 256)
    o[i] = El<T>::st(i < W ? f(late(i)) : 0.f);
}

// cast of [x | x0] with zero padding
template <typename T>
__global__ void __launch_bounds__(256)
k_cat_rows(const float* __restrict__ x, const float* __restrict__ x0,
           T* __restrict__ out, int W, int Kp) {
  const size_t r = blockIdx.x;
#pragma unroll 8
  for (int i = threadIdx.x; i < Kp; i += 256)
    out[r * Kp + i] = El<T>::st(
        i < W ? x[r * W + i] : i < 2 * W ? x0[r * W + i - W] : 0.f);
}

// ---- one row: y[n] = W[n] . staged row, one wave per NR outputs ----------
// The row is staged into LDS as T: normed or convolved (stage_row),
// concatenated [x | x0], through the polynomial activation, from several
// streams (stage_hyper) or normed in parts; block 0 can persist it to hout,
// and the residual to xout.  A row that is T already (hin) is read where it
// lies; there blockIdx.y picks one of up to two products.  A wave always has
// its next slab of weights on the way, the first one during the staging.
enum { EPI_F32 = 0, EPI_RESADD = 1, EPI_SOFTCAP = 2, EPI_T = 3, EPI_TGATE = 4,
       EPI_RELU2 = 5, EPI_ROTARY = 6, EPI_GELU = 7 };
enum { ROW_NORM = 0, ROW_CAT = 1, ROW_PLAIN = 2, ROW_CONV = 3, ROW_POLY = 4,
       ROW_HYPER = 5, ROW_GROUPS = 6 };

struct LinRowArgs {
  const void* Wt;           // [N, Kp]
  RowStage s;               // ROW_CAT: xadd is the second half
  const int* rows;          // nullable: source row
  const void* hin;          // ROW_PLAIN
  void* hout;               // nullable
  const float* bias;        // nullable
  const float* act;         // ROW_POLY: four coefficients; the row is s.x
  void* y;                  // fp32, or T for EPI_RELU2 and EPI_GELU
  int N, stage, epi;
  float cap;
  int groups;               // ROW_GROUPS
  int Z, K2;                // ROW_PLAIN: products, and K of the second,
  long xz, wz, yz;          // which lies this many elements further on
  HyperStage h;             // ROW_HYPER (s has W and Kp, too)
};

DEVINL float relu2_f(float v) {
  v = fmaxf(v, 0.f);
  return v * v;
}
DEVINL float gelu_f(float v) {
  return 0.5f * v * (1.f + erff(v * 0.7071067811865476f));
}

#define LIN_NT 512
template <typename T, int MODE, int U, int NR, int HS = 0>
__global__ void __launch_bounds__(LIN_NT) k_lin_row(LinRowArgs a) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  __shared__ float red[LIN_NT / 64 * (MODE == ROW_POLY ? 3 : 1)];
  constexpr int V = El<T>::V, S = 64 * V, NK = 8 / NR;
  T* xs = (T*)smem;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int z = MODE == ROW_PLAIN ? blockIdx.y : 0;
  const int N = a.N, Kp = z ? a.K2 : a.s.Kp;
  const T* Wt = (const T*)a.Wt + (MODE == ROW_PLAIN ? z * a.wz : 0);
  const int step = gridDim.x * (LIN_NT / 64) * NR;
  int n = (blockIdx.x * (LIN_NT / 64) + wave) * NR, k0 = 0;
  f4v w[NR][NK], next[NR][NK];
  auto slab = [&](f4v (&to)[NR][NK], int n0, int kb) {
#pragma unroll
    for (int i = 0; i < NR; i++) {
      const T* wr = Wt + (size_t)min(n0 + i, N - 1) * Kp;
#pragma unroll
      for (int u = 0; u < NK; u++) {
        const int k = kb + u * S + lane * V;
        to[i][u] = k < Kp ? ld16nt(wr + k) : f4v{0.f, 0.f, 0.f, 0.f};
      }
    }
  };
  slab(w, n, 0);
  const size_t row = a.rows ? a.rows[0] : 0;
  const bool first = blockIdx.x == 0;
  if constexpr (MODE == ROW_NORM || MODE == ROW_CONV) {
    stage_row<LIN_NT, U, MODE == ROW_CONV>(a.s, row, first, red,
                                           [&](int i, float f) {
      T v = El<T>::st(f);
      xs[i] = v;
      if (a.hout && first) ((T*)a.hout)[i] = v;
    });
  } else if constexpr (MODE == ROW_HYPER) {
    stage_hyper<LIN_NT, U, HS>(a.h, row, first, red, [&](int i, float f) {
      T v = El<T>::st(f);
      xs[i] = v;
      if (a.hout && first) ((T*)a.hout)[i] = v;
    });
  } else if constexpr (MODE == ROW_GROUPS) {
    stage_groups<LIN_NT>(a.s, a.groups, row, (float*)(xs + Kp),
                         [&](int i, float f) { xs[i] = El<T>::st(f); });
  } else if constexpr (MODE == ROW_POLY) {
    const int W = a.s.W;
    const float* z = a.s.x + row * W;
    float v[U];
#pragma unroll
    for (int u = 0; u < U; u++) {
      const int i = tid + u * LIN_NT;
      v[u] = i < W ? z[i] : 0.f;
    }
    auto late = [&](int i) { return z[i]; };
    const PolyNorm f = poly_moments<LIN_NT, U>(v, late, W, a.act, a.s.eps, red);
#pragma unroll
    for (int u = 0; u < U; u++) {
      const int i = tid + u * LIN_NT;
      if (i < Kp) xs[i] = El<T>::st(i < W ? f(v[u]) : 0.f);
    }
    for (int i = tid + U * LIN_NT; i < Kp; i += LIN_NT)
      xs[i] = El<T>::st(i < W ? f(late(i)) : 0.f);
  } else if constexpr (MODE == ROW_CAT) {
    const int W = a.s.W;
    const float *x = a.s.x + row * W, *x0 = a.s.xadd + row * W;
    for (int i = tid; i < Kp; i += LIN_NT)
      xs[i] = El<T>::st(i < W ? x[i] : i < 2 * W ? x0[i - W] : 0.f);
  }
  const T* xr = MODE == ROW_PLAIN ? (const T*)a.hin + z * a.xz : xs;
  if (MODE != ROW_PLAIN) __syncthreads();
  float acc[NR];
#pragma unroll
  for (int i = 0; i < NR; i++) acc[i] = 0.f;
  while (n < N) {
    int n1 = n, k1 = k0 + NK * S;
    if (k1 >= Kp) {
      k1 = 0;
      n1 += step;
    }
    if (n1 < N) slab(next, n1, k1);
#pragma unroll
    for (int u = 0; u < NK; u++) {
      const int k = k0 + u * S + lane * V;
      if (k < Kp) {
        f4v xv = ld16(xr + k);
#pragma unroll
        for (int i = 0; i < NR; i++) acc[i] = dot16<T>(w[i][u], xv, acc[i]);
      }
    }
    if (k1 == 0)
#pragma unroll
      for (int i = 0; i < NR; i++) {
        float v = wave_reduce_sum(acc[i]);
        acc[i] = 0.f;
        if (lane == 0 && n + i < N) {
          if (a.bias) v += a.bias[n + i];
          if (a.cap > 0.f) v = a.cap * tanhf(v / a.cap);
          if (a.epi == EPI_RELU2) ((T*)a.y)[n + i] = El<T>::st(relu2_f(v));
          else if (a.epi == EPI_GELU) ((T*)a.y)[n + i] = El<T>::st(gelu_f(v));
          else if (MODE == ROW_PLAIN) ((float*)a.y)[z * a.yz + n + i] = v;
          else ((float*)a.y)[n + i] = v;
        }
      }
#pragma unroll
    for (int i = 0; i < NR; i++)
#pragma unroll
      for (int u = 0; u < NK; u++) w[i][u] = next[i][u];
    n = n1;
    k0 = k1;
  }
}

// ---- many rows: MFMA GEMM ---------------------------------------------
// EPI_ROTARY: columns from `split` on are heads of RT values, of which the
// first `dims` rotate in pairs (2i, 2i+1); they go to y[row*ld + head*hs].
struct Rotary {
  const int* pos;
  const float *cosT, *sinT;   // [positions, dims/2]
  void* y;
  int split, RT, dims, ld, hs;
};

struct GemmArgs {
  const void *X, *W;
  void* Y;
  const float* gate;        // EPI_TGATE: sigmoid(gate[row*ldg + z*gz + col*gc])
  const float* bias;        // nullable: added per column
  int M, N, K, ldx, ldw, ldy, ldg, epi, gz, gc;
  float mult;               // EPI_RESADD multiplier / EPI_SOFTCAP cap
  long xz, wz, yz;          // per-z (head) element offsets
  int K2;                   // K, and ldw, of z > 0
  struct Rotary r;          // EPI_ROTARY
};

template <typename T, int EPI>
DEVINL void gemm_store(const GemmArgs& a, int z, int row, int col, float v) {
  const size_t o = (size_t)z * a.yz + (size_t)row * a.ldy + col;
  if (row >= a.M || col >= a.N) return;
  if constexpr (EPI == EPI_F32) ((float*)a.Y)[o] = v;
  else if constexpr (EPI == EPI_RESADD) ((float*)a.Y)[o] += a.mult * v;
  else if constexpr (EPI == EPI_SOFTCAP)
    ((float*)a.Y)[o] = a.mult > 0.f ? a.mult * tanhf(v / a.mult) : v;
  else if constexpr (EPI == EPI_T) ((T*)a.Y)[o] = El<T>::st(v);
  else if constexpr (EPI == EPI_RELU2) ((T*)a.Y)[o] = El<T>::st(relu2_f(v));
  else if constexpr (EPI == EPI_GELU) ((T*)a.Y)[o] = El<T>::st(gelu_f(v));
  else
    ((T*)a.Y)[o] = El<T>::st(
        v * sigmoid_f(a.gate[(size_t)row * a.ldg + z * a.gz + col * a.gc]));
}

// the same for NR consecutive rows, v[r] of row0 + r
template <typename T, int EPI, int NR>
DEVINL void gemm_store_rows(const GemmArgs& a, int z, int row0, int col,
                            const float* v) {
  if constexpr (EPI != EPI_ROTARY) {
#pragma unroll
    for (int r = 0; r < NR; r++)
      gemm_store<T, EPI>(a, z, row0 + r, col, v[r]);
  } else {
    // every lane of the wave comes here, neighbours with neighbouring columns
    const Rotary& t = a.r;
    const int c = max(col - t.split, 0), h = c / t.RT, j = c - h * t.RT;
    const bool rot = col >= t.split, turn = rot && j < t.dims;
    float cs[NR], sn[NR], other[NR];
    if (__any(turn))
#pragma unroll
      for (int r = 0; r < NR; r++) {
        const size_t k = (size_t)t.pos[min(row0 + r, a.M - 1)] * (t.dims >> 1) +
                         (turn ? j >> 1 : 0);
        cs[r] = t.cosT[k];
        sn[r] = t.sinT[k];
      }
#pragma unroll
    for (int r = 0; r < NR; r++) other[r] = __shfl_xor(v[r], 1);
#pragma unroll
    for (int r = 0; r < NR; r++) {
      const int row = row0 + r;
      const float o =
          turn ? v[r] * cs[r] + (j & 1 ? other[r] : -other[r]) * sn[r] : v[r];
      T* to = rot ? (T*)t.y + (size_t)row * t.ld + (size_t)h * t.hs + j
                  : (T*)a.Y + (size_t)row * a.ldy + col;
      if (row < a.M && col < a.N) *to = El<T>::st(o);
    }
  }
}

// run body(integral constant of the epilogue)
template <class Body> DEVINL void with_epilogue(int epi, Body body) {
  switch (epi) {
    case EPI_F32: body(std::integral_constant<int, EPI_F32>()); break;
    case EPI_RESADD: body(std::integral_constant<int, EPI_RESADD>()); break;
    case EPI_SOFTCAP: body(std::integral_constant<int, EPI_SOFTCAP>()); break;
    case EPI_T: body(std::integral_constant<int, EPI_T>()); break;
    case EPI_TGATE: body(std::integral_constant<int, EPI_TGATE>()); break;
    case EPI_RELU2: body(std::integral_constant<int, EPI_RELU2>()); break;
    case EPI_ROTARY: body(std::integral_constant<int, EPI_ROTARY>()); break;
    case EPI_GELU: body(std::integral_constant<int, EPI_GELU>()); break;
  }
}

template <typename T, int BM, int BN>
__global__ void __launch_bounds__(256) k_gemm(GemmArgs a) {
  __shared__ __attribute__((aligned(16))) char lds[gemm_lds_bytes<BM, BN>()];
  const int bm = blockIdx.y * BM, bn = blockIdx.x * BN, z = blockIdx.z;
  const T* X = (const T*)a.X + (size_t)z * a.xz;
  const T* W = (const T*)a.W + (size_t)z * a.wz;
  const int K = z ? a.K2 : a.K, ldw = z ? a.K2 : a.ldw;
  f4v acc[BM / 32][BN / 32];
  gemm_mainloop<BM, BN, T>(
      acc, lds,
      [&](int r) { return X + (size_t)min(bm + r, a.M - 1) * a.ldx; },
      [&](int r) { return W + (size_t)min(bn + r, a.N - 1) * ldw; }, 0,
      K / GemmMma<T>::BK);
  float bias[BN / 32];
#pragma unroll
  for (int j = 0; j < BN / 32; j++)
    bias[j] = a.bias ? a.bias[min(bn + gemm_col<BN>(j), a.N - 1)] : 0.f;
  with_epilogue(a.epi, [&](auto epi) {
#pragma unroll
    for (int i = 0; i < BM / 32; i++)
#pragma unroll
      for (int j = 0; j < BN / 32; j++) {
        const int col = bn + gemm_col<BN>(j);
        float v[4];
#pragma unroll
        for (int r = 0; r < 4; r++) v[r] = acc[i][j][r] + bias[j];
        gemm_store_rows<T, decltype(epi)::value, 4>(
            a, z, bm + gemm_row0<BM>(i), col, v);
      }
  });
}

// up to 16*MF rows: a tile of NB (16, or 8 to have more blocks) outputs per
// block, K over NW waves, both operands straight from memory (the weights are
// read once)
template <typename T, int MF, int NW, int NB = 16>
__global__ void __launch_bounds__(64 * NW) k_gemm_skinny(GemmArgs a) {
  __shared__ float red[NW * MF * 256];
  constexpr int U = MF == 1 ? 8 : 4;
  const int tid = threadIdx.x, wave = wave_index(), lane = tid & 63;
  const int lr = lane & 15, gq = lane >> 4, z = blockIdx.z;
  const int K = z ? a.K2 : a.K, ldw = z ? a.K2 : a.ldw;
  const int n0 = blockIdx.x * NB, nch = K * (int)sizeof(T) / 64;
  const char* wr = (const char*)((const T*)a.W + (size_t)z * a.wz +
                                 (size_t)min(n0 + lr, a.N - 1) * ldw) +
                   gq * 16;
  const char* xr[MF];
#pragma unroll
  for (int i = 0; i < MF; i++)
    xr[i] = (const char*)((const T*)a.X + (size_t)z * a.xz +
                          (size_t)min(i * 16 + lr, a.M - 1) * a.ldx) + gq * 16;
  f4v acc[MF];
#pragma unroll
  for (int i = 0; i < MF; i++) acc[i] = {0.f, 0.f, 0.f, 0.f};
  for (int c = wave; c < nch; c += U * NW) {
    f4v w[U], xv[U][MF];
#pragma unroll
    for (int u = 0; u < U; u++) {
      const int cu = c + u * NW;
      const bool in = cu < nch;
      w[u] = in && lr < NB ? ld16nt(wr + (size_t)cu * 64) : f4v{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < MF; i++)
        xv[u][i] = in ? ld16(xr[i] + cu * 64) : f4v{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll
    for (int u = 0; u < U; u++)
#pragma unroll
      for (int i = 0; i < MF; i++)
        acc[i] = GemmMma<T>::mma(xv[u][i], w[u], acc[i]);
  }
#pragma unroll
  for (int i = 0; i < MF; i++)
#pragma unroll
    for (int r = 0; r < 4; r++)
      red[(wave * MF + i) * 256 + (gq * 4 + r) * 16 + lr] = acc[i][r];
  __syncthreads();
  for (int e = tid; e < MF * 256; e += 64 * NW) {
    float v = 0.f;
#pragma unroll
    for (int u = 0; u < NW; u++) v += red[u * MF * 256 + e];
    const int row = e >> 4, col = (e & 15) < NB ? n0 + (e & 15) : a.N;
    if (a.bias) v += a.bias[min(col, a.N - 1)];
    with_epilogue(a.epi, [&](auto epi) {
      gemm_store_rows<T, decltype(epi)::value, 1>(a, z, row, col, &v);
    });
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

extern "C" hipError_t launch_embed_pairs(int f32, const PairEmbed* a,
                                         hipStream_t s) {
  if (a->M < 1 || a->W < 1 || a->S < 1 || a->nd < 0 || a->nd > a->M ||
      a->nseg < 0 || a->buckets < 1 || a->mul_before < 0 || a->mul_cur < 0)
    return hipErrorInvalidValue;
  BY_TYPE(f32,
          hipLaunchKernelGGL(k_embed_pairs<u16>, dim3(a->M), dim3(256), 0, s, *a),
          hipLaunchKernelGGL(k_embed_pairs<float>, dim3(a->M), dim3(256), 0, s,
                             *a));
  if (a->nseg)
    hipLaunchKernelGGL(k_last_tokens, dim3((a->nseg + 255) / 256), dim3(256), 0,
                       s, *a);
  return hipGetLastError();
}

static bool bad_hyper(const HyperStage& s) {
  return s.W < 1 || s.S < 1 || s.S > MAX_STREAMS || !s.x || !s.in != !s.g ||
         (s.in && s.Kp < s.W) || (s.y && (!s.mix || !s.feed)) ||
         (s.y2 && (!s.y || !s.gb || !s.gb2)) || (!s.in && !s.xout);
}

template <typename T, int U>
static void hyper_go(const HyperStage& s, const int* rows, T* out, int M,
                     hipStream_t st) {
  if (s.S == 2)
    hipLaunchKernelGGL((k_hyper_rows<T, U, 2>), dim3(M), dim3(256), 0, st, s,
                       rows, out);
  else if (s.S == 4)
    hipLaunchKernelGGL((k_hyper_rows<T, U, 4>), dim3(M), dim3(256), 0, st, s,
                       rows, out);
  else
    hipLaunchKernelGGL((k_hyper_rows<T, 1, 0>), dim3(M), dim3(256), 0, st, s,
                       rows, out);
}

extern "C" hipError_t launch_hyper_rows(int f32, const HyperStage* s,
                                        const void* rows, void* out, int M,
                                        hipStream_t st) {
  if (bad_hyper(*s) || M < 1 || (s->in && !out) || (s->xout && rows))
    return hipErrorInvalidValue;
  const int* r = (const int*)rows;
  if (s->W <= 2048)
    BY_TYPE(f32, (hyper_go<u16, 8>(*s, r, (u16*)out, M, st)),
            (hyper_go<float, 8>(*s, r, (float*)out, M, st)));
  else
    BY_TYPE(f32, (hyper_go<u16, 16>(*s, r, (u16*)out, M, st)),
            (hyper_go<float, 16>(*s, r, (float*)out, M, st)));
  return hipGetLastError();
}

static bool bad_groups(const RowStage& s, int groups) {
  return s.W < 1 || !s.x || !s.g || s.Kp < s.W || groups < 1 ||
         groups > MAX_GROUPS || s.W % groups;
}

extern "C" hipError_t launch_group_rows(int f32, const RowStage* s, int groups,
                                        void* out, int M, hipStream_t st) {
  if (bad_groups(*s, groups) || M < 1) return hipErrorInvalidValue;
  BY_TYPE(f32,
          hipLaunchKernelGGL(k_group_rows<u16>, dim3(M), dim3(256), 0, st, *s,
                             groups, (u16*)out),
          hipLaunchKernelGGL(k_group_rows<float>, dim3(M), dim3(256), 0, st, *s,
                             groups, (float*)out));
  return hipGetLastError();
}

static bool bad_stage(const RowStage& s) {
  return s.W < 1 || !s.x || !s.y != !s.gb || (s.g && s.Kp < s.W) ||
         (s.gate && s.ldg < s.W);
}

template <typename T>
static void norm_rows(const RowStage& s, const void* rows, void* out, int M,
                      hipStream_t st) {
  if (s.W <= 2048)
    hipLaunchKernelGGL((k_norm_rows<T, 8>), dim3(M), dim3(256), 0, st, s,
                       (const int*)rows, (T*)out);
  else
    hipLaunchKernelGGL((k_norm_rows<T, 16>), dim3(M), dim3(256), 0, st, s,
                       (const int*)rows, (T*)out);
}

extern "C" hipError_t launch_norm_rows(int f32, const RowStage* s,
                                       const void* rows, void* out, int M,
                                       hipStream_t st) {
  if (bad_stage(*s) || M < 1 || (!s->g && !s->xout) || (s->xout && rows))
    return hipErrorInvalidValue;
  if (f32) norm_rows<float>(*s, rows, out, M, st);
  else norm_rows<u16>(*s, rows, out, M, st);
  return hipGetLastError();
}

static bool bad_conv(const RowStage& s) {
  return bad_stage(s) || !s.cw || !s.ring || !s.slot || !s.pos || s.taps < 1 ||
         s.Kp < s.W || s.xadd || s.g || s.gate || (s.y && !s.xout);
}

template <typename T, int NT, int R>
static void conv_go(const ConvRows& a, hipStream_t st) {
  const dim3 grid(a.nd + a.nchunk * (CHUNK / R));
#define CONV_TAPS(n)                                                         \
  case n:                                                                    \
    hipLaunchKernelGGL((k_conv_rows<T, n, NT, R>), grid, dim3(NT), 0, st, a); \
    break
  switch (a.s.taps) {
    CONV_TAPS(1);
    CONV_TAPS(2);
    CONV_TAPS(3);
    CONV_TAPS(4);
  }
#undef CONV_TAPS
}

template <typename T>
static hipError_t conv_rows(const ConvRows& a, hipStream_t st) {
  const int W = a.s.W;
  if (a.s.taps <= 4 && W % 4 == 0 && W <= 4096) {
    if (W <= 1024)
      a.nchunk ? conv_go<T, 256, 4>(a, st) : conv_go<T, 256, 1>(a, st);
    else if (W <= 2048)
      a.nchunk ? conv_go<T, 512, 4>(a, st) : conv_go<T, 512, 1>(a, st);
    else
      a.nchunk ? conv_go<T, 1024, 4>(a, st) : conv_go<T, 1024, 1>(a, st);
  } else {
    const size_t lds = (ANY_R + a.s.taps - 1) * sizeof(float);
    hipLaunchKernelGGL(k_conv_rows_any<T>,
                       dim3(a.nd + a.nchunk * (CHUNK / ANY_R)), dim3(256), lds,
                       st, a);
    hipLaunchKernelGGL(k_conv_ring, dim3(a.nd + a.nseg), dim3(256), 0, st, a,
                       a.s.xout ? a.s.xout : a.s.x);
  }
  return hipGetLastError();
}

extern "C" hipError_t launch_conv_rows(int f32, const ConvRows* a,
                                       hipStream_t st) {
  if (bad_conv(a->s) || a->s.xout == a->s.x || !a->out || a->nd < 0 ||
      a->nchunk < 0 || a->nd + a->nchunk < 1 || !a->nseg != !a->nchunk ||
      a->s.Kp % 64 || a->s.Kp >= a->s.W + 64 ||
      a->s.taps > 8192)
    return hipErrorInvalidValue;
  return f32 ? conv_rows<float>(*a, st) : conv_rows<u16>(*a, st);
}

template <typename T>
static void poly_rows(const void* z, int ldz, const void* coef, void* out,
                      int M, int W, int Kp, float eps, hipStream_t s) {
  if (W <= 4096)
    hipLaunchKernelGGL((k_poly_rows<T, 16>), dim3(M), dim3(256), 0, s,
                       (const float*)z, ldz, (const float*)coef, (T*)out, W,
                       Kp, eps);
  else
    hipLaunchKernelGGL((k_poly_rows<T, 40>), dim3(M), dim3(256), 0, s,
                       (const float*)z, ldz, (const float*)coef, (T*)out, W,
                       Kp, eps);
}

extern "C" hipError_t launch_poly_rows(int f32, const void* z, int ldz,
                                       const void* coef, void* out, int M,
                                       int W, int Kp, float eps,
                                       hipStream_t s) {
  if (M < 1 || W < 1 || Kp < W || ldz < W) return hipErrorInvalidValue;
  if (f32) poly_rows<float>(z, ldz, coef, out, M, W, Kp, eps, s);
  else poly_rows<u16>(z, ldz, coef, out, M, W, Kp, eps, s);
  return hipGetLastError();
}

extern "C" hipError_t launch_cat_rows(int f32, const void* x, const void* x0,
                                      void* out, int M, int W, int Kp,
                                      hipStream_t s) {
  if (M < 1 || Kp < 2 * W) return hipErrorInvalidValue;
  BY_TYPE(f32,
          hipLaunchKernelGGL(k_cat_rows<u16>, dim3(M), dim3(256), 0, s,
                             (const float*)x, (const float*)x0, (u16*)out, W,
                             Kp),
          hipLaunchKernelGGL(k_cat_rows<float>, dim3(M), dim3(256), 0, s,
                             (const float*)x, (const float*)x0, (float*)out,
                             W, Kp));
  return hipGetLastError();
}

template <typename T, int MODE, int U, int NR, int HS>
static hipError_t lin_row_nr(const LinRowArgs& a, hipStream_t s) {
  constexpr int per = LIN_NT / 64 * NR;
  RAISE_LDS((k_lin_row<T, MODE, U, NR, HS>));
  int blocks = (a.N + per - 1) / per;
  const int rounds = (blocks + 511) / 512;       // alike in every block
  blocks = (blocks + rounds - 1) / rounds;
  size_t lds = MODE == ROW_PLAIN ? 0 : (size_t)a.s.Kp * sizeof(T);
  if (MODE == ROW_GROUPS) lds += MAX_GROUPS * sizeof(float);   // sums of parts
  hipLaunchKernelGGL((k_lin_row<T, MODE, U, NR, HS>),
                     dim3(blocks, MODE == ROW_PLAIN ? a.Z : 1), dim3(LIN_NT),
                     lds, s, a);
  return hipGetLastError();
}

template <typename T, int MODE, int U, int HS = 0>
static hipError_t lin_row_go(const LinRowArgs& a, hipStream_t s) {
  return a.N <= 4096 ? lin_row_nr<T, MODE, U, 1, HS>(a, s)
                     : lin_row_nr<T, MODE, U, 2, HS>(a, s);
}

template <typename T>
static hipError_t lin_row(const LinRowArgs& a, hipStream_t s) {
  if (a.N < 1 || a.s.Kp < 64 || a.s.Kp % 64 ||
      (a.epi != EPI_F32 && a.epi != EPI_RELU2 && a.epi != EPI_GELU))
    return hipErrorInvalidValue;
  if (a.Z < 1 || a.Z > 2 ||
      (a.Z == 2 && (a.stage != ROW_PLAIN || a.K2 < 64 || a.K2 % 64 ||
                    a.epi != EPI_F32)))
    return hipErrorInvalidValue;
  if (a.stage == ROW_PLAIN)
    return a.hin ? lin_row_go<T, ROW_PLAIN, 1>(a, s) : hipErrorInvalidValue;
  if ((size_t)a.s.Kp * sizeof(T) > 150 * 1024) return hipErrorInvalidValue;
  if (a.stage == ROW_CAT)
    return a.s.xadd && a.s.Kp >= 2 * a.s.W ? lin_row_go<T, ROW_CAT, 1>(a, s)
                                           : hipErrorInvalidValue;
  if (a.stage == ROW_POLY) {
    if (!a.s.x || !a.act || a.s.W < 1 || a.s.Kp < a.s.W)
      return hipErrorInvalidValue;
    return a.s.W <= 4096 ? lin_row_go<T, ROW_POLY, 8>(a, s)
                         : lin_row_go<T, ROW_POLY, 20>(a, s);
  }
  if (a.stage == ROW_CONV) {
    if (bad_conv(a.s) || a.s.xout == a.s.x || a.rows)
      return hipErrorInvalidValue;
    return a.s.W <= 2048 ? lin_row_go<T, ROW_CONV, 4>(a, s)
                         : lin_row_go<T, ROW_CONV, 8>(a, s);
  }
  if (a.stage == ROW_GROUPS)
    return bad_groups(a.s, a.groups) ? hipErrorInvalidValue
                                     : lin_row_go<T, ROW_GROUPS, 1>(a, s);
  // other blocks read x while block 0 writes xout
  if (a.stage == ROW_HYPER) {
    const HyperStage& h = a.h;
    if (bad_hyper(h) || !h.in || h.xout == h.x || h.W != a.s.W ||
        h.Kp != a.s.Kp)
      return hipErrorInvalidValue;
    if (h.S == 2)
      return h.W <= 2048 ? lin_row_go<T, ROW_HYPER, 4, 2>(a, s)
                         : lin_row_go<T, ROW_HYPER, 8, 2>(a, s);
    if (h.S == 4)
      return h.W <= 2048 ? lin_row_go<T, ROW_HYPER, 4, 4>(a, s)
                         : lin_row_go<T, ROW_HYPER, 8, 4>(a, s);
    return lin_row_go<T, ROW_HYPER, 1, 0>(a, s);
  }
  if (a.stage != ROW_NORM || bad_stage(a.s) || !a.s.g || a.s.xout == a.s.x) return hipErrorInvalidValue;
  return a.s.W <= 2048 ? lin_row_go<T, ROW_NORM, 4>(a, s)
                       : lin_row_go<T, ROW_NORM, 8>(a, s);
}

extern "C" hipError_t launch_lin_row(int f32, const LinRowArgs* a,
                                     hipStream_t s) {
  return f32 ? lin_row<float>(*a, s) : lin_row<u16>(*a, s);
}

template <typename T>
static void gemm_go(const GemmArgs& a, int Z, hipStream_t s) {
  long b128 = (long)((a.M + 127) / 128) * ((a.N + 127) / 128) * Z;
  dim3 sk((a.N + 15) / 16, 1, Z);
  if (a.M <= 16 && sk.x * Z <= 128 && a.K >= 4096) {   // few blocks, deep K
    hipLaunchKernelGGL((k_gemm_skinny<T, 1, 16, 8>), dim3((a.N + 7) / 8, 1, Z),
                       dim3(1024), 0, s, a);
  } else if (a.M <= 16 && sk.x * Z <= 256 && a.K >= 4096) {
    hipLaunchKernelGGL((k_gemm_skinny<T, 1, 16>), sk, dim3(1024), 0, s, a);
  } else if (a.M <= 16) {
    hipLaunchKernelGGL((k_gemm_skinny<T, 1, 8>), sk, dim3(512), 0, s, a);
  } else if (a.M <= 32) {
    hipLaunchKernelGGL((k_gemm_skinny<T, 2, 8>), sk, dim3(512), 0, s, a);
  } else if (a.M <= 64) {
    hipLaunchKernelGGL((k_gemm_skinny<T, 4, 8>), sk, dim3(512), 0, s, a);
  } else if (b128 < 192) {
    hipLaunchKernelGGL((k_gemm<T, 64, 64>),
                       dim3((a.N + 63) / 64, (a.M + 63) / 64, Z), dim3(256), 0,
                       s, a);
  } else if (b128 < 300 || b128 < 0.7 * 512 * ((b128 + 511) / 512)) {
    // two 128x128 tiles fit a CU; a part-filled last wave of them is worse
    hipLaunchKernelGGL((k_gemm<T, 128, 64>),
                       dim3((a.N + 63) / 64, (a.M + 127) / 128, Z), dim3(256),
                       0, s, a);
  } else {
    hipLaunchKernelGGL((k_gemm<T, 128, 128>),
                       dim3((a.N + 127) / 128, (a.M + 127) / 128, Z),
                       dim3(256), 0, s, a);
  }
}

extern "C" hipError_t launch_gemm_rows(int f32, const void* X, const void* W,
                                       void* Y, const void* gate,
                                       const void* bias, int M,
                                       int N, int K, int ldx, int ldw,
                                       int ldy, int ldg, int epi, float mult,
                                       int Z, long xz, long wz, long yz,
                                       int gz, int gc, const Rotary* rotary,
                                       int K2, hipStream_t s) {
  if (M < 1 || N < 1 || K < 64 || K % 64 || ldx < K || ldw < K || Z < 1 ||
      K2 < 64 || K2 % 64 || ldx < K2 ||
      epi < 0 || epi > EPI_GELU || (epi == EPI_TGATE && !gate))
    return hipErrorInvalidValue;
  GemmArgs a = {X, W, Y, (const float*)gate, (const float*)bias, M, N, K, ldx,
                ldw, ldy, ldg, epi, gz, gc, mult, xz, wz, yz, K2, {}};
  if (epi == EPI_ROTARY) {
    if (!rotary || rotary->split % 2 || rotary->RT < 2 || rotary->RT % 2 ||
        rotary->dims % 2 || rotary->dims > rotary->RT || Z != 1 ||
        (N - rotary->split) % rotary->RT)
      return hipErrorInvalidValue;
    a.r = *rotary;
  }
  if (f32) gemm_go<float>(a, Z, s);
  else gemm_go<u16>(a, Z, s);
  return hipGetLastError();
}
