// Grouped-query attention whose key weights are sigmoids, over a paged cache
// of rows [keys (kvh * dim) | values (kvh * vdim)].
//
// The projections of a token pass a causal convolution of ``taps`` per
// channel; queries and keys then an RMS norm per head. The last ``taps``
// projected rows of a sequence are kept in its state, that of position p at
// p % taps, so that a decode step can write its own without touching one that
// another block of the step reads.
//
// With z = scale q.k - r1 ln(1 + r2 distance) + pb the weight of a key is
// 1 / (1 + exp(-z)). Weights are not normalized, so there is no running
// maximum and partial results of a split simply add.
//
// Both attention kernels compute the scores transposed (keys along a lane's
// registers, queries or heads along the lanes): the weights then lie in the
// registers as the second matrix product reads them, with its keys in the
// order 4 lg + j, 16 + 4 lg + j (j < 4) within 32, lg = lane / 16.
//
// T is u16 (bfloat16 bits) or float. Scores, weights and sums are float32; a
// weight enters a bfloat16 product as a high and a low part.
#include "fei_attn.h"

namespace {

struct Geo {           // sizes of one mixer
  int heads, kvh, dim, vdim;
  float scale;
  int window;          // keys a query sees, itself included; 0 = all
};

struct Conv {
  const float* w;      // [taps][channels]
  const float* qn;     // [dim]
  const float* kn;     // [dim]
  int taps;
  float eps;
};

__device__ __forceinline__ int channels(const Geo& g) {
  return g.heads * g.dim + g.kvh * (g.dim + g.vdim);
}

// Per-head norm of a group's LG x 8 values of which n count.
template <int LG>
__device__ __forceinline__ void head_norm(float (&y)[8], int n, float eps,
                                          const float (&wn)[8]) {
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < 8; ++j) ss = fmaf(y[j], y[j], ss);
  ss = row16_sum(ss);
  if (LG == 32) ss += __shfl_xor(ss, 16);
  const float inv = 1.f / sqrtf(ss / (float)n + eps);
#pragma unroll
  for (int j = 0; j < 8; ++j) y[j] *= inv * wn[j];
}

// Convolution and norms of prompt rows: queries to q, keys and values to
// their cache rows. A group of LG lanes takes one head of RUN rows one after
// another, a lane 8 of its channels: the weights and the TAPS - 1 projections
// before a row stay in registers. spans [.][3]: first row, rows, first
// position. Sizes are multiples of 8.
constexpr int RUN = 8;

template <typename T, int LG, int TAPS>
__global__ void __launch_bounds__(256)
k_sig_conv_run(T* __restrict__ q, const T* __restrict__ proj, long ps,
               T* __restrict__ rows, const float* __restrict__ states,
               Conv cv, const int* __restrict__ spans,
               const int* __restrict__ row_seq, const int* __restrict__ pos,
               const int* __restrict__ slots, const int* __restrict__ table,
               int n_rows, int seq0, int W, int bs_log, Geo g) {
  const int units = g.heads + 2 * g.kvh;
  const int item = blockIdx.x * (256 / LG) + threadIdx.x / LG;
  const int t0 = item / units * RUN, u = item % units;
  if (t0 >= n_rows) return;                // whole groups
  const int CH = channels(g), R = g.kvh * (g.dim + g.vdim);
  const bool is_q = u < g.heads, is_v = u >= g.heads + g.kvh;
  const int n = is_v ? g.vdim : g.dim;
  const int ch0 = is_v ? (g.heads + g.kvh) * g.dim +
                             (u - g.heads - g.kvh) * g.vdim
                       : u * g.dim;
  const int c = (threadIdx.x & (LG - 1)) * 8;
  const bool on = c < n;
  const int ch = ch0 + (on ? c : 0);
  float w[TAPS][8], wn[8], past[TAPS][8];  // past[a]: a rows back; [0] unused
#pragma unroll
  for (int i = 0; i < TAPS; ++i) {
    const f32x8 v = ld8(cv.w + (long)i * CH + ch);
#pragma unroll
    for (int j = 0; j < 8; ++j) w[i][j] = v[j];
  }
  if (!is_v) {
    const f32x8 v = ld8((is_q ? cv.qn : cv.kn) + (on ? c : 0));
#pragma unroll
    for (int j = 0; j < 8; ++j) wn[j] = v[j];
  }
  int last = -1;
#pragma unroll
  for (int k = 0; k < RUN; ++k) {
    const int t = t0 + k;
    if (t >= n_rows) return;
    const int row = seq0 + t, seq = row_seq[row], p = pos[row];
    if (seq != last) {                     // the run or a portion starts
      last = seq;
      const int row0 = spans[(seq - seq0) * 3];
#pragma unroll
      for (int a = 1; a < TAPS; ++a) {
        if (row - a >= row0) {
          const auto v = ld8(proj + (long)(row - a) * ps + ch);
#pragma unroll
          for (int j = 0; j < 8; ++j) past[a][j] = get8(v, j);
        } else if (p - a >= 0) {
          const f32x8 v = ld8(states + ((long)slots[seq] * TAPS +
                                        (p - a) % TAPS) * CH + ch);
#pragma unroll
          for (int j = 0; j < 8; ++j) past[a][j] = v[j];
        } else {
#pragma unroll
          for (int j = 0; j < 8; ++j) past[a][j] = 0.f;
        }
      }
    }
    const auto v = ld8(proj + (long)row * ps + ch);
    float y[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const float x = get8(v, j);
      y[j] = 0.f;
#pragma unroll
      for (int a = TAPS - 1; a > 0; --a)
        y[j] = fmaf(w[TAPS - 1 - a][j], past[a][j], y[j]);
      y[j] = on ? fmaf(w[TAPS - 1][j], x, y[j]) : 0.f;
#pragma unroll
      for (int a = TAPS - 1; a > 1; --a) past[a][j] = past[a - 1][j];
      if (TAPS > 1) past[TAPS > 1 ? 1 : 0][j] = x;
    }
    if (!is_v) head_norm<LG>(y, n, cv.eps, wn);
    if (on) {
      T* dst = is_q ? q + (long)t * g.heads * g.dim + ch
                    : rows + cache_row(table, W, seq, p, bs_log) * R +
                          (ch - g.heads * g.dim);
      typename El<T>::frag o;
#pragma unroll
      for (int j = 0; j < 8; ++j) o[j] = El<T>::st(y[j]);
      st8(dst, o);
    }
  }
}

// The same for any sizes and any number of taps, one row per group.
template <typename T, int LG, bool VEC>
__global__ void __launch_bounds__(256)
k_sig_conv(T* __restrict__ q, const T* __restrict__ proj, long ps,
           T* __restrict__ rows, const float* __restrict__ states, Conv cv,
           const int* __restrict__ spans, const int* __restrict__ row_seq,
           const int* __restrict__ pos, const int* __restrict__ slots,
           const int* __restrict__ table, int n_rows, int seq0, int W,
           int bs_log, Geo g) {
  const int units = g.heads + 2 * g.kvh;
  const int item = blockIdx.x * (256 / LG) + threadIdx.x / LG;
  if (item >= n_rows * units) return;      // whole groups
  const int t = item / units, u = item - t * units;
  const int row = seq0 + t, seq = row_seq[row], p = pos[row];
  const int row0 = spans[(seq - seq0) * 3];
  const int CH = channels(g);
  const bool is_v = u >= g.heads + g.kvh;
  const int n = is_v ? g.vdim : g.dim;
  const int ch0 = is_v ? (g.heads + g.kvh) * g.dim +
                             (u - g.heads - g.kvh) * g.vdim
                       : u * g.dim;
  const int c = (threadIdx.x & (LG - 1)) * 8;
  const float* st = states ? states + (long)slots[seq] * cv.taps * CH : nullptr;
  float y[8];
#pragma unroll
  for (int j = 0; j < 8; ++j) y[j] = 0.f;
  if (c < n) {
    for (int i = 0; i < cv.taps; ++i) {
      const int a = cv.taps - 1 - i;
      if (p - a < 0) continue;
      const float* wt = cv.w + (long)i * CH + ch0 + c;
      if (row - a >= row0) {
        const T* src = proj + (long)(row - a) * ps + ch0 + c;
        if (VEC) {
          const auto v = ld8(src);
          const auto w = ld8(wt);
#pragma unroll
          for (int j = 0; j < 8; ++j) y[j] = fmaf(w[j], get8(v, j), y[j]);
        } else {
#pragma unroll
          for (int j = 0; j < 8; ++j)
            if (c + j < n) y[j] = fmaf(wt[j], El<T>::ld(src[j]), y[j]);
        }
      } else {
        const float* src = st + (long)((p - a) % cv.taps) * CH + ch0 + c;
#pragma unroll
        for (int j = 0; j < 8; ++j)
          if (c + j < n) y[j] = fmaf(wt[j], src[j], y[j]);
      }
    }
  }
  if (!is_v) {
    const float* src = u < g.heads ? cv.qn : cv.kn;
    float wn[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) wn[j] = c + j < n ? src[c + j] : 0.f;
    head_norm<LG>(y, n, cv.eps, wn);
  }
  if (c >= n) return;
  T* dst = u < g.heads
               ? q + (long)t * g.heads * g.dim + ch0 + c
               : rows + cache_row(table, W, seq, p, bs_log) *
                            (g.kvh * (g.dim + g.vdim)) +
                     (ch0 - g.heads * g.dim) + c;
  if (VEC) {
    typename El<T>::frag o;
#pragma unroll
    for (int j = 0; j < 8; ++j) o[j] = El<T>::st(y[j]);
    st8(dst, o);
  } else {
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (c + j < n) dst[j] = El<T>::st(y[j]);
  }
}

// State after the portions: their last projected rows. grid (portions, taps,
// ceil(channels / 256))
template <typename T>
__global__ void __launch_bounds__(256)
k_sig_state(float* __restrict__ states, const T* __restrict__ proj, long ps,
            const int* __restrict__ spans, const int* __restrict__ slots,
            int seq0, int taps, int CH) {
  const int* sp = spans + blockIdx.x * 3;
  const int a = blockIdx.y, n = sp[1];
  if (a >= n) return;
  const int p = sp[2] + n - 1 - a;
  const T* src = proj + (long)(sp[0] + n - 1 - a) * ps;
  const int i = blockIdx.z * 256 + threadIdx.x;
  if (i < CH)
    states[((long)slots[seq0 + blockIdx.x] * taps + p % taps) * CH + i] =
        El<T>::ld(src[i]);
}

// Place of a key of a tile of 64 in the order of the second product.
__device__ __forceinline__ int key_place(int key) {
  return (key & 32) + ((key & 15) >> 2) * 8 + ((key >> 4) & 1) * 4 + (key & 3);
}

// Attention of prompt portions. grid (heads, query tiles, 128 / (16 NW QS)); a
// wave owns QS sets of 16 queries, which share the fragments it reads, the
// block walks the keys they see in tiles of 64 held in LDS: keys row-major,
// values transposed. The distance bias depends on query - key alone: a tile's
// NW * 16 * QS + 63 values are computed once, in four copies shifted by one
// each, so that a lane reads the four of its keys as one aligned vector.
// KS >= ceil(dim / 32), DC >= ceil(vdim / 16); queries are zero beyond dim,
// columns beyond vdim are not stored.
template <typename T, int KS, int DC, int NW, int QS, bool VEC>
__global__ void __launch_bounds__(NW * 64, 2)
k_sig_prefill(T* __restrict__ out, long os, const T* __restrict__ q,
              const T* __restrict__ rows, const float* __restrict__ bias,
              const int* __restrict__ spans, const int* __restrict__ tiles,
              const int* __restrict__ table, int seq0, int W, int bs_log,
              Geo g) {
  typedef typename El<T>::frag frag;
  constexpr int NP = Parts<T>::n;
  constexpr int NT = NW * 64, NQ = NW * 16 * QS;
  constexpr int DS = KS * 32 + 8;          // odd count of 16-byte slots
  constexpr int TB = NQ + 68;
  extern __shared__ __align__(16) char smem[];
  T* kt = (T*)smem;                        // [64][DS]
  T* vt = kt + 64 * DS;                    // [DC * 16][64], see vt_at
  float* tb = (float*)(vt + DC * 16 * 64);  // [4][TB]

  const int h = blockIdx.x, gk = h / (g.heads / g.kvh);
  // a portion's last queries see the most keys: they start first
  const int tile = gridDim.y - 1 - blockIdx.y;
  const int pt = tiles[tile * 2];
  const int row0 = spans[pt * 3], cnt = spans[pt * 3 + 1];
  const int pos0 = spans[pt * 3 + 2];
  const int q0 = tiles[tile * 2 + 1] + blockIdx.z * NQ;
  if (q0 >= cnt) return;
  const int qn = min(NQ, cnt - q0);
  const int tid = threadIdx.x, lane = tid & 63;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l15 = lane & 15, lg = lane >> 4;
  const int R = g.kvh * (g.dim + g.vdim);
  const T* kh = rows + (long)gk * g.dim;
  const T* vh = rows + (long)g.kvh * g.dim + (long)gk * g.vdim;

  frag bq[QS][KS];
  f32x4 o[QS][DC];
#pragma unroll
  for (int i = 0; i < QS; ++i) {
    const int r = min((w * QS + i) * 16 + l15, qn - 1);
    const T* src = q + (long)(row0 - seq0 + q0 + r) * g.heads * g.dim +
                   (long)h * g.dim;
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      const int c = k * 32 + 8 * lg;
#pragma unroll
      for (int j = 0; j < 8; ++j) bq[i][k][j] = 0;
      if (VEC) {
        if (c < g.dim) bq[i][k] = ld8(src + c);
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j)
          if (c + j < g.dim) bq[i][k][j] = src[c + j];
      }
    }
#pragma unroll
    for (int d = 0; d < DC; ++d) o[i][d] = f32x4{0.f, 0.f, 0.f, 0.f};
  }

  // positions of this tile's queries and of the keys any of them sees
  const int qa = pos0 + q0, qb = qa + qn - 1;
  const int klo = first_key(qa, g.window) & ~63;
  // this wave's own range: tiles outside it are staged for the others only
  const int wa = qa + w * 16 * QS, wb = min(wa + 16 * QS - 1, qb);
  const int wlo = first_key(wa, g.window);
  const float r1 = bias[h], r2 = bias[g.heads + h], pb = bias[2 * g.heads + h];
  const float scale = -g.scale * El<T>::base;
  const unsigned seen = g.window > 0 ? g.window : 1u << 31;

  // Cached rows of a tile's keys. Keys past the last query are read as that
  // query's own: their weights are zero, their values have to be finite.
  const int seq = seq0 + pt;
  auto tile_row = [&](int t0) {
    return bs_log >= 6 ? cache_row(table, W, seq, t0, bs_log) : 0L;
  };
  auto row_of = [&](long first, int t0, int r) {
    const int key = min(t0 + r, qb);
    return bs_log >= 6 ? first + (key - t0)
                       : cache_row(table, W, seq, key, bs_log);
  };
  // vector loads of a tile: all of them before the first store
  constexpr int NV = KS * 4, NC = DC * 2;
  constexpr int UK = (64 * NV + NT - 1) / NT, UV = (32 * NC + NT - 1) / NT;
  frag kf[UK], va[UV], vb[UV];
  auto load = [&](int t0) {
    const long first = tile_row(t0);
#pragma unroll
    for (int u = 0; u < UK; ++u) {
      const int i = tid + u * NT;
      const int r = i / NV, c = (i - r * NV) * 8;
      kf[u] = ld8(kh + row_of(first, t0, r & 63) * R + (c < g.dim ? c : 0));
    }
#pragma unroll
    for (int u = 0; u < UV; ++u) {
      const int i = tid + u * NT;
      const int r = (i / NC * 2) & 63, c = min(i % NC * 8, g.vdim - 8);
      va[u] = ld8(vh + row_of(first, t0, r) * R + c);
      vb[u] = ld8(vh + row_of(first, t0, r + 1) * R + c);
    }
  };
  if (VEC) load(klo);

  for (int t0 = klo; t0 <= qb; t0 += 64) {
    __syncthreads();
    if (VEC) {
#pragma unroll
      for (int u = 0; u < UK; ++u) {
        const int i = tid + u * NT;
        const int r = i / NV, c = (i - r * NV) * 8;
        if (64 * NV % NT == 0 || i < 64 * NV) st8(kt + r * DS + c, kf[u]);
      }
#pragma unroll
      for (int u = 0; u < UV; ++u) {
        const int i = tid + u * NT;
        const int r = key_place(i / NC * 2), c = i % NC * 8;
        if (32 * NC % NT == 0 || i < 32 * NC)
#pragma unroll
          for (int j = 0; j < 8; ++j) {
            T two[2] = {(T)va[u][j], (T)vb[u][j]};
            __builtin_memcpy(vt + vt_at(c + j, r), two, sizeof(two));
          }
      }
    } else {
      const long first = tile_row(t0);
      for (int i = tid; i < 64 * KS * 32; i += NT) {
        const int r = i / (KS * 32), c = i - r * (KS * 32);
        kt[r * DS + c] = c < g.dim ? kh[row_of(first, t0, r) * R + c]
                                   : El<T>::st(0.f);
      }
      for (int i = tid; i < 64 * DC * 16; i += NT) {
        const int r = i / (DC * 16), c = i - r * (DC * 16);
        vt[vt_at(c, key_place(r))] = c < g.vdim
                                         ? vh[row_of(first, t0, r) * R + c]
                                         : El<T>::st(0.f);
      }
    }
    for (int i = tid; i < NQ + 63; i += NT) {
      const int d = max(qa - t0 + NQ - 1 - i, 0);
      const float v = (r1 * El<T>::ln(1.f + r2 * (float)d) - pb) * El<T>::base;
#pragma unroll
      for (int s = 0; s < 4; ++s)
        if (i >= s) tb[s * TB + i - s] = v;
    }
    __syncthreads();
    if (VEC && t0 + 64 <= qb) load(t0 + 64);
    if (t0 > wb || t0 + 63 < wlo) continue;

    f32x4 s[QS][4];
#pragma unroll
    for (int c = 0; c < 4; ++c) {
#pragma unroll
      for (int i = 0; i < QS; ++i) s[i][c] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < KS; ++k) {
        const frag a = ld8(kt + (c * 16 + l15) * DS + k * 32 + 8 * lg);
#pragma unroll
        for (int i = 0; i < QS; ++i) s[i][c] = mma(a, bq[i][k], s[i][c]);
      }
    }
    // no mask where every query of the wave sees every key of the tile
    const bool edge = t0 + 63 > wa || (g.window > 0 && wb - t0 >= g.window);
    const int sh = (3 - l15) & 3;
#pragma unroll
    for (int i = 0; i < QS; ++i) {
      const int qp = wa + i * 16 + l15;
      const float* tq = tb + sh * TB + 4 * lg - (w * QS + i) * 16 - l15 + NQ -
                        1 - sh;
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        const f32x4 b = *(const f32x4*)(tq + c * 16);
#pragma unroll
        for (int r = 0; r < 4; ++r)
          s[i][c][r] =
              El<T>::inv(1.f + El<T>::exb(fmaf(s[i][c][r], scale, b[r])));
      }
      if (edge) {
        const int d0 = qp - t0 - 4 * lg;
#pragma unroll
        for (int c = 0; c < 4; ++c)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const unsigned d = d0 - c * 16 - r;   // a key ahead: huge
            if (d >= seen) s[i][c][r] = 0.f;
          }
      }
    }
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      frag pw[QS][NP];
#pragma unroll
      for (int i = 0; i < QS; ++i) {
        float v[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) v[j] = s[i][2 * k + (j >> 2)][j & 3];
        weight_parts(v, pw[i]);
      }
#pragma unroll
      for (int d = 0; d < DC; ++d) {
        const frag av = ld8(vt + vt_at(d * 16 + l15, k * 32 + 8 * lg));
#pragma unroll
        for (int i = 0; i < QS; ++i)
#pragma unroll
          for (int n = 0; n < NP; ++n) o[i][d] = mma(av, pw[i][n], o[i][d]);
      }
    }
  }

#pragma unroll
  for (int i = 0; i < QS; ++i) {
    const int r = (w * QS + i) * 16 + l15;
    if (r >= qn) continue;
    T* dst = out + (long)(row0 + q0 + r) * os + (long)h * g.vdim;
#pragma unroll
    for (int d = 0; d < DC; ++d) {
      const int c = d * 16 + 4 * lg;
      T v[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = El<T>::st(o[i][d][j]);
      if (VEC) {
        if (c < g.vdim) __builtin_memcpy(dst + c, v, sizeof(v));
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (c + j < g.vdim) dst[c + j] = v[j];
      }
    }
  }
}

// Keys of a decode row in splits: base (a multiple of 32), keys per split.
__device__ __forceinline__ void split_of(int p, int window, int splits,
                                         int least, int* base, int* chunk) {
  *base = first_key(p, window) & ~31;
  const int n = p + 1 - *base;
  *chunk = ((n + splits - 1) / splits + least - 1) / least * least;
}

// Decode: one token of each sequence, from its projections to attention
// outputs. grid (splits, kvh * ceil(group / 16), B); a block takes the keys of
// one split for up to 16 heads that share a key/value head, a wave 32 keys at
// a time. Every block makes the queries of its heads; the one whose split
// ends with the new token also makes its key and value, writes its cache row
// and reads them from LDS. Split 0 writes the state.
// A lane holds CPL value columns: CPL * 16 >= vdim. KS >= ceil(dim / 32).
template <typename T, int KS, int CPL, bool VEC>
__global__ void
__launch_bounds__(256, sizeof(T) == 2 && KS <= 4 && CPL <= 8 ? 2 : 1)
k_sig_decode(T* __restrict__ out, long os, float* __restrict__ part,
             const T* __restrict__ proj, long ps, T* __restrict__ rows,
             float* __restrict__ states, Conv cv,
             const float* __restrict__ bias, const int* __restrict__ pos,
             const int* __restrict__ slots, const int* __restrict__ table,
             int W, int bs_log, Geo g, int splits, int least) {
  typedef typename El<T>::frag frag;
  constexpr int NP = Parts<T>::n;
  constexpr int DS = KS * 32 + 8;
  constexpr int VS = CPL * 16;             // value columns of the lanes
  extern __shared__ __align__(16) char smem[];
  T* qs = (T*)smem;                        // [16][DS]
  T* kn = qs + 16 * DS;                    // [DS]
  T* vn = kn + DS;                         // [VS]
  float* red = (float*)(vn + VS);          // [4][heads of the block][VS + 4]

  const int split = blockIdx.x, b = blockIdx.z;
  const int hg = g.heads / g.kvh, ht = (hg + 15) / 16;
  const int gk = blockIdx.y / ht, hy = blockIdx.y - gk * ht;
  const int h0 = gk * hg + hy * 16, nh = min(16, hg - hy * 16);
  const int tid = threadIdx.x, w = tid >> 6, lane = tid & 63;
  const int l15 = lane & 15, lg = lane >> 4;
  const int R = g.kvh * (g.dim + g.vdim), CH = channels(g);
  const int p = pos[b], k0 = first_key(p, g.window);
  int base, chunk;
  split_of(p, g.window, splits, least, &base, &chunk);
  const int lo = base + split * chunk, hi = min(lo + chunk, p + 1);
  if (lo > p) return;
  const bool owner = hi == p + 1;
  const T* kh = rows + (long)gk * g.dim;
  const T* vh = rows + (long)g.kvh * g.dim + (long)gk * g.vdim;

  struct Tile {
    frag k[2][KS];
    T v[8][CPL];
  };
  auto key_of = [&](int it, int j) {       // key of value register j
    return it + (j < 4 ? 4 * lg + j : 12 + 4 * lg + j);
  };
  auto load = [&](Tile& t, int it) {
    const long first = bs_log >= 5 ? cache_row(table, W, b, it, bs_log) : 0L;
    auto row_of = [&](int key) {
      key = min(key, p);                   // beyond p: replaced, see below
      return bs_log >= 5 ? first + (key - it)
                         : cache_row(table, W, b, key, bs_log);
    };
#pragma unroll
    for (int c = 0; c < 2; ++c) {
      const T* src = kh + row_of(it + c * 16 + l15) * R;
#pragma unroll
      for (int k = 0; k < KS; ++k) {
        const int col = k * 32 + 8 * lg;
        if (VEC) {
          t.k[c][k] = ld8(src + (col < g.dim ? col : 0));
        } else {
#pragma unroll
          for (int j = 0; j < 8; ++j)
            t.k[c][k][j] = src[col + j < g.dim ? col + j : 0];
        }
      }
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const T* src = vh + row_of(key_of(it, j)) * R;
      const int col = l15 * CPL;
      if (VEC) {
        constexpr int N = CPL < 8 ? CPL : 8;
#pragma unroll
        for (int i = 0; i < CPL; i += N)
          __builtin_memcpy(&t.v[j][i],
                           __builtin_assume_aligned(
                               src + (col + i < g.vdim ? col + i : 0),
                               N * sizeof(T) < 16 ? N * sizeof(T) : 16),
                           N * sizeof(T));
      } else {
#pragma unroll
        for (int i = 0; i < CPL; ++i)
          t.v[j][i] = src[col + i < g.vdim ? col + i : 0];
      }
    }
  };
  int it = lo + 32 * w;
  Tile cur;
  if (it < hi) load(cur, it);

  // queries of the block's heads, then the new key and value
  {
    float* st = states ? states + (long)slots[b] * cv.taps * CH : nullptr;
    const T* pr = proj + (long)b * ps;
    const int newest = p % cv.taps;
    auto ring = [&](int a) {               // place of the row a positions back
      const int i = newest - a;
      return i < 0 ? i + cv.taps : i;
    };
    const int units = owner || split == 0 ? nh + 2 : nh;
    for (int u = w; u < units; u += 4) {
      const bool is_q = u < nh, is_v = u == nh + 1;
      const int n = is_v ? g.vdim : g.dim;
      const int ch0 = is_q ? (h0 + u) * g.dim
                           : g.heads * g.dim +
                                 (is_v ? g.kvh * g.dim + gk * g.vdim
                                       : gk * g.dim);
      const bool keep = st && split == 0 && (is_q || hy == 0);
      // all loads of up to 4 taps before the first use
      float x[4][4], cw[4][4], y[4], ss = 0.f;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int c = lane + 64 * i;
        if (c < n) {
          x[i][0] = El<T>::ld(pr[ch0 + c]);
          cw[i][0] = cv.w[(long)(cv.taps - 1) * CH + ch0 + c];
#pragma unroll
          for (int a = 1; a < 4; ++a) {
            x[i][a] = cw[i][a] = 0.f;
            if (a < cv.taps && a <= p) {
              x[i][a] = st[(long)ring(a) * CH + ch0 + c];
              cw[i][a] = cv.w[(long)(cv.taps - 1 - a) * CH + ch0 + c];
            }
          }
        }
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int c = lane + 64 * i;
        y[i] = 0.f;
        if (c < n) {
          for (int a = min(cv.taps - 1, p); a >= 4; --a)
            y[i] = fmaf(cv.w[(long)(cv.taps - 1 - a) * CH + ch0 + c],
                        st[(long)ring(a) * CH + ch0 + c], y[i]);
#pragma unroll
          for (int a = 3; a >= 0; --a) y[i] = fmaf(cw[i][a], x[i][a], y[i]);
          if (keep) st[(long)ring(0) * CH + ch0 + c] = x[i][0];
          ss = fmaf(y[i], y[i], ss);
        }
      }
      if (!is_q && !owner) continue;
      float inv = 1.f;
      if (!is_v) inv = 1.f / sqrtf(wave_reduce_sum(ss) / (float)n + cv.eps);
      const float* wn = is_q ? cv.qn : cv.kn;
      T* dst = is_q ? qs + u * DS : is_v ? vn : kn;
      T* row = rows + cache_row(table, W, b, p, bs_log) * R +
               (ch0 - g.heads * g.dim);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int c = lane + 64 * i;
        if (c < (is_v ? VS : KS * 32)) {
          const T v = El<T>::st(c < n ? y[i] * inv * (is_v ? 1.f : wn[c])
                                      : 0.f);
          dst[c] = v;
          if (!is_q && hy == 0 && c < n) row[c] = v;
        }
      }
    }
  }
  __syncthreads();
  frag bq[KS];
#pragma unroll
  for (int k = 0; k < KS; ++k) {
    bq[k] = ld8(qs + min(l15, nh - 1) * DS + k * 32 + 8 * lg);
    if (l15 >= nh) {
#pragma unroll
      for (int j = 0; j < 8; ++j) bq[k][j] = 0;
    }
  }
  const int hb = h0 + min(l15, nh - 1);
  const float r1 = bias[hb], r2 = bias[g.heads + hb];
  const float pb = bias[2 * g.heads + hb];
  const float scale = -g.scale * El<T>::base;
  f32x4 acc[CPL];
#pragma unroll
  for (int i = 0; i < CPL; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};

  for (; it < hi; it += 128) {
    Tile nxt;
    if (it + 128 < hi) load(nxt, it + 128);
    if (it + 31 >= p) {      // the new token's row, and none beyond it
#pragma unroll
      for (int c = 0; c < 2; ++c)
        if (it + c * 16 + l15 >= p) {
#pragma unroll
          for (int k = 0; k < KS; ++k)
            cur.k[c][k] = ld8(kn + k * 32 + 8 * lg);
        }
#pragma unroll
      for (int j = 0; j < 8; ++j)
        if (key_of(it, j) >= p) {
#pragma unroll
          for (int i = 0; i < CPL; ++i) cur.v[j][i] = vn[l15 * CPL + i];
        }
    }
    frag pw[NP];
    float pv[8];
#pragma unroll
    for (int c = 0; c < 2; ++c) {
      f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < KS; ++k) s = mma(cur.k[c][k], bq[k], s);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = it + c * 16 + 4 * lg + r;
        const float d = (float)max(p - key, 0);
        const float off = (r1 * El<T>::ln(1.f + r2 * d) - pb) * El<T>::base;
        float v = El<T>::inv(1.f + El<T>::exb(fmaf(s[r], scale, off)));
        if (key > p || key < k0) v = 0.f;
        pv[c * 4 + r] = v;
      }
    }
    weight_parts(pv, pw);
#pragma unroll
    for (int i = 0; i < CPL; ++i) {
      frag av;
#pragma unroll
      for (int j = 0; j < 8; ++j) av[j] = cur.v[j][i];
#pragma unroll
      for (int n = 0; n < NP; ++n) acc[i] = mma(av, pw[n], acc[i]);
    }
    cur = nxt;
  }

  if (l15 < nh) {
    float* dst = red + ((long)w * nh + l15) * (VS + 4);
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int i = 0; i < CPL; ++i) dst[(4 * lg + r) * CPL + i] = acc[i][r];
  }
  __syncthreads();
  const int step = nh * (VS + 4);
  for (int i = tid; i < nh * g.vdim; i += 256) {
    const int h = i / g.vdim, c = i - h * g.vdim;
    const float* x = red + h * (VS + 4) + c;
    const float v = (x[0] + x[step]) + (x[2 * step] + x[3 * step]);
    const int col = (h0 + h) * g.vdim + c;
    if (splits == 1)
      out[(long)b * os + col] = El<T>::st(v);
    else
      part[((long)b * splits + split) * g.heads * g.vdim + col] = v;
  }
}

// Sum of the splits that had keys. grid (ceil(heads * vdim / 256), B)
template <typename T>
__global__ void __launch_bounds__(256)
k_sig_combine(T* __restrict__ out, long os, const float* __restrict__ part,
              const int* __restrict__ pos, int window, int splits, int least,
              int HV) {
  const int c = blockIdx.x * 256 + threadIdx.x, b = blockIdx.y;
  if (c >= HV) return;
  const int p = pos[b];
  int base, chunk;
  split_of(p, window, splits, least, &base, &chunk);
  const int n = (p + 1 - base + chunk - 1) / chunk;
  const float* x = part + (long)b * splits * HV + c;
  float v = 0.f;
  int s = 0;
  for (; s + 4 <= n; s += 4)
    v += (x[(long)s * HV] + x[(long)(s + 1) * HV]) +
         (x[(long)(s + 2) * HV] + x[(long)(s + 3) * HV]);
  for (; s < n; ++s) v += x[(long)s * HV];
  out[(long)b * os + c] = El<T>::st(v);
}

template <typename K>
void allow_lds(K kernel) {
  (void)hipFuncSetAttribute((const void*)kernel,
                            hipFuncAttributeMaxDynamicSharedMemorySize,
                            160 * 1024);
}

template <typename T>
void run_decode(T* out, long os, float* part, const T* proj, long ps, T* rows,
                float* states, Conv cv, const float* bias, const int* pos,
                const int* slots, const int* table, int B, int W, int bs_log,
                Geo g, int splits, int least, hipStream_t stream) {
  const int hg = g.heads / g.kvh;
  const dim3 grid(splits, g.kvh * ((hg + 15) / 16), B);
  const bool vec = g.dim % 8 == 0 && g.vdim % 8 == 0;
#define DEC(KS, CPL, VEC)                                                    \
  do {                                                                       \
    static bool set = false;                                                 \
    if (!set) {                                                              \
      allow_lds(k_sig_decode<T, KS, CPL, VEC>);                              \
      set = true;                                                            \
    }                                                                        \
    const size_t lds = sizeof(T) * (17 * (KS * 32 + 8) + CPL * 16) +         \
                       4 * 4 * (hg < 16 ? hg : 16) * (CPL * 16 + 4);         \
    hipLaunchKernelGGL((k_sig_decode<T, KS, CPL, VEC>), grid, dim3(256),     \
                       lds, stream, out, os, part, proj, ps, rows, states,   \
                       cv, bias, pos, slots, table, W, bs_log, g, splits,    \
                       least);                                               \
  } while (0)
#define BY_CPL(KS)                                \
  do {                                            \
    if (g.vdim <= 64) DEC(KS, 4, true);           \
    else if (g.vdim <= 128) DEC(KS, 8, true);     \
    else DEC(KS, 16, true);                       \
  } while (0)
  if (!vec) DEC(8, 16, false);
  else if (g.dim <= 64) BY_CPL(2);
  else if (g.dim <= 128) BY_CPL(4);
  else BY_CPL(8);
#undef BY_CPL
#undef DEC
  if (splits > 1) {
    const int HV = g.heads * g.vdim;
    hipLaunchKernelGGL(k_sig_combine<T>, dim3((HV + 255) / 256, B), dim3(256),
                       0, stream, out, os, part, pos, g.window, splits, least,
                       HV);
  }
}

template <typename T>
void run_conv(T* q, const T* proj, long ps, T* rows, float* states, Conv cv,
              const int* spans, const int* row_seq, const int* pos,
              const int* slots, const int* table, int n_rows, int seq0,
              int n_portions, int W, int bs_log, Geo g, hipStream_t stream) {
  const bool vec = g.dim % 8 == 0 && g.vdim % 8 == 0 && ps % 8 == 0;
  const long items = (long)n_rows * (g.heads + 2 * g.kvh);
  const bool small = g.dim <= 128 && g.vdim <= 128;
#define CONV(LG, VEC)                                                        \
  hipLaunchKernelGGL((k_sig_conv<T, LG, VEC>),                               \
                     dim3((items + 256 / LG - 1) / (256 / LG)), dim3(256),   \
                     0, stream, q, proj, ps, rows, states, cv, spans,        \
                     row_seq, pos, slots, table, n_rows, seq0, W, bs_log, g)
#define CONV_RUN(LG, TAPS)                                                   \
  hipLaunchKernelGGL((k_sig_conv_run<T, LG, TAPS>),                          \
                     dim3((runs + 256 / LG - 1) / (256 / LG)), dim3(256), 0, \
                     stream, q, proj, ps, rows, states, cv, spans, row_seq,  \
                     pos, slots, table, n_rows, seq0, W, bs_log, g)
#define BY_LG(TAPS)                                              \
  do {                                                           \
    if (small) CONV_RUN(16, TAPS); else CONV_RUN(32, TAPS);      \
  } while (0)
  const long runs = (long)((n_rows + RUN - 1) / RUN) *
                    (g.heads + 2 * g.kvh);
  if (vec && cv.taps == 1) BY_LG(1);
  else if (vec && cv.taps == 2) BY_LG(2);
  else if (vec && cv.taps == 3) BY_LG(3);
  else if (vec && cv.taps == 4) BY_LG(4);
  else if (small && vec) CONV(16, true);
  else if (small) CONV(16, false);
  else if (vec) CONV(32, true);
  else CONV(32, false);
#undef BY_LG
#undef CONV_RUN
#undef CONV
  const int CH = g.heads * g.dim + g.kvh * (g.dim + g.vdim);
  if (states)
    hipLaunchKernelGGL(k_sig_state<T>,
                       dim3(n_portions, cv.taps, (CH + 255) / 256), dim3(256),
                       0, stream, states, proj, ps, spans, slots, seq0,
                       cv.taps, CH);
}

template <typename T, int KS, int DC, bool VEC>
void launch_prefill(T* out, long os, const T* q, const T* rows,
                    const float* bias, const int* spans, const int* tiles,
                    const int* table, int n_tiles, int seq0, int W, int bs_log,
                    Geo g, hipStream_t stream) {
  // the registers of two sets of queries suffice up to these sizes
  constexpr int QS = sizeof(T) == 2 && KS <= 4 && DC <= 8 ? 2 : 1;
  constexpr int NW = sizeof(T) == 2 ? 8 / QS : 4;
  constexpr int NQ = NW * 16 * QS;
  static bool set = false;
  if (!set) {
    allow_lds(k_sig_prefill<T, KS, DC, NW, QS, VEC>);
    set = true;
  }
  const size_t lds = sizeof(T) * (64 * (KS * 32 + 8) + DC * 16 * 64) +
                     16 * (NQ + 68);
  const dim3 grid(g.heads, n_tiles, 128 / NQ);
  hipLaunchKernelGGL((k_sig_prefill<T, KS, DC, NW, QS, VEC>), grid,
                     dim3(NW * 64), lds, stream, out, os, q, rows, bias,
                     spans, tiles, table, seq0, W, bs_log, g);
}

template <typename T>
void run_prefill(T* out, long os, const T* q, const T* rows,
                 const float* bias, const int* spans, const int* tiles,
                 const int* table, int n_tiles, int seq0, int W, int bs_log,
                 Geo g, hipStream_t stream) {
#define PRE(KS, DC, VEC)                                                     \
  launch_prefill<T, KS, DC, VEC>(out, os, q, rows, bias, spans, tiles,       \
                                 table, n_tiles, seq0, W, bs_log, g, stream)
#define BY_DC(KS)                             \
  do {                                        \
    if (g.vdim <= 64) PRE(KS, 4, true);       \
    else if (g.vdim <= 128) PRE(KS, 8, true); \
    else PRE(KS, 16, true);                   \
  } while (0)
  if (g.dim % 8 || g.vdim % 8 || os % 4) PRE(8, 16, false);
  else if (g.dim <= 64) BY_DC(2);
  else if (g.dim <= 128) BY_DC(4);
  else BY_DC(8);
#undef BY_DC
#undef PRE
}

}  // namespace

extern "C" {

// taps == 1: states may be null.
void fei_sig_decode(void* out, long os, float* part, const void* proj, long ps,
                    void* rows, float* states, const float* conv,
                    const float* qn, const float* kn, const float* bias,
                    const int* pos, const int* slots, const int* table, int B,
                    int W, int bs_log, int heads, int kvh, int dim, int vdim,
                    int taps, int window, float scale, int splits, float eps,
                    int least, int f32, hipStream_t stream) {
  const Geo g{heads, kvh, dim, vdim, scale, window};
  const Conv cv{conv, qn, kn, taps, eps};
  if (f32)
    run_decode<float>((float*)out, os, part, (const float*)proj, ps,
                      (float*)rows, states, cv, bias, pos, slots, table, B, W,
                      bs_log, g, splits, least, stream);
  else
    run_decode<u16>((u16*)out, os, part, (const u16*)proj, ps, (u16*)rows,
                    states, cv, bias, pos, slots, table, B, W, bs_log, g,
                    splits, least, stream);
}

void fei_sig_conv(void* q, const void* proj, long ps, void* rows,
                  float* states, const float* conv, const float* qn,
                  const float* kn, const int* spans, const int* row_seq,
                  const int* pos, const int* slots, const int* table,
                  int n_rows, int seq0, int n_portions, int W, int bs_log,
                  int heads, int kvh, int dim, int vdim, int taps, float eps,
                  int f32, hipStream_t stream) {
  const Geo g{heads, kvh, dim, vdim, 1.f, 0};
  const Conv cv{conv, qn, kn, taps, eps};
  if (f32)
    run_conv<float>((float*)q, (const float*)proj, ps, (float*)rows, states,
                    cv, spans, row_seq, pos, slots, table, n_rows, seq0,
                    n_portions, W, bs_log, g, stream);
  else
    run_conv<u16>((u16*)q, (const u16*)proj, ps, (u16*)rows, states, cv,
                  spans, row_seq, pos, slots, table, n_rows, seq0, n_portions,
                  W, bs_log, g, stream);
}

void fei_sig_prefill(void* out, long os, const void* q, const void* rows,
                     const float* bias, const int* spans, const int* tiles,
                     const int* table, int n_tiles, int seq0, int W,
                     int bs_log, int heads, int kvh, int dim, int vdim,
                     int window, float scale, int f32, hipStream_t stream) {
  const Geo g{heads, kvh, dim, vdim, scale, window};
  if (f32)
    run_prefill<float>((float*)out, os, (const float*)q, (const float*)rows,
                       bias, spans, tiles, table, n_tiles, seq0, W, bs_log, g,
                       stream);
  else
    run_prefill<u16>((u16*)out, os, (const u16*)q, (const u16*)rows, bias,
                     spans, tiles, table, n_tiles, seq0, W, bs_log, g, stream);
}

}  // extern "C"
