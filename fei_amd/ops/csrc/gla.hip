// Gated linear attention: per head a state S [vdim][dim] (value-major),
//   S_t = S_(t-1) * diag(alpha_t) + v_t k_t^T,   o_t = S_t q_t,
// with a decay alpha per key channel, alpha = sigmoid(z)^(1/tau), z a low-rank
// map of the input. Everything past the projections is float32, matrix
// products included (float32 MFMA).
//
// Prompts go by chunks of 64 tokens. With G_t the sum of log decays from the
// chunk's start through t, a chunk with start state S gives
//   o_t = (q_t exp(G_t)) S + sum_{s<=t} A_ts v_s,
//   A_ts = sum_d q_td k_sd exp(G_td - G_sd),
//   S' = S diag(exp(G_end)) + sum_s v_s (k_s exp(G_end - G_s))^T.
// No exponent is positive anywhere (A goes by blocks of 16 tokens: within a
// block term by term, between blocks relative to the later block's start), so
// decays may be arbitrarily strong.
//   k_gla_gate    G
//   k_gla_state   each chunk's own sum for S'
//   k_gla_scan    start state of every chunk, last state into the slot
//   k_gla_scores  A
//   k_gla_out     o, head norm, output gate
// Decode: k_gla_decode updates the state and reads it, k_gla_gate_out norms.
//
// A projected row is [q (H dim) | k (H dim) | v (H vdim) | gate (H vdim) |
// decay input (rank)]; T is u16 (bfloat16 bits) or float.
#include "fei_common.h"
#include "fei_mma.h"

namespace {

constexpr int CH = 64;       // tokens per chunk

struct Gla {
  int heads, dim, vdim, rank;
  float tau;
  __device__ __host__ int kq() const { return heads * dim; }
  __device__ __host__ int vo() const { return heads * vdim; }
  __device__ __host__ int k_off() const { return kq(); }
  __device__ __host__ int v_off() const { return 2 * kq(); }
  __device__ __host__ int g_off() const { return 2 * kq() + vo(); }
  __device__ __host__ int a_off() const { return 2 * kq() + 2 * vo(); }
};

__device__ __forceinline__ float log_decay(float z, float inv_tau) {
  return (fminf(z, 0.f) - log1pf(expf(-fabsf(z)))) * inv_tau;
}

// chunks [.][3]: portion, first row, rows. G [T][H dim].
// grid (chunks, ceil(H dim / 64)): 64 channels x 4 groups of 16 tokens.
template <typename T>
__global__ void __launch_bounds__(256)
k_gla_gate(float* __restrict__ G, const T* __restrict__ proj, long ps,
           const float* __restrict__ a2, const float* __restrict__ bias,
           const int* __restrict__ chunks, Gla g) {
  extern __shared__ float as[];            // [rank][CH]
  __shared__ float tot[4][64];
  const int row0 = chunks[blockIdx.x * 3 + 1], n = chunks[blockIdx.x * 3 + 2];
  for (int i = threadIdx.x; i < CH * g.rank; i += 256) {
    const int t = i / g.rank, r = i - t * g.rank;
    as[r * CH + t] = t < n ? El<T>::ld(proj[(long)(row0 + t) * ps + g.a_off() + r])
                           : 0.f;
  }
  __syncthreads();
  const float inv_tau = 1.f / g.tau;
  const int cx = threadIdx.x & 63, sb = threadIdx.x >> 6;
  const int c = blockIdx.y * 64 + cx;
  float z[16];
  if (c < g.kq()) {
    const float b = bias[c];
#pragma unroll
    for (int t = 0; t < 16; ++t) z[t] = b;
    for (int r = 0; r < g.rank; ++r) {
      const float w = a2[(long)c * g.rank + r];
#pragma unroll
      for (int t = 0; t < 16; ++t) z[t] = fmaf(w, as[r * CH + sb * 16 + t], z[t]);
    }
    float sum = 0.f;
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      sum += log_decay(z[t], inv_tau);
      z[t] = sum;
    }
    tot[sb][cx] = sum;
  }
  __syncthreads();
  if (c < g.kq()) {
    float off = 0.f;
    for (int i = 0; i < sb; ++i) off += tot[i][cx];
#pragma unroll
    for (int t = 0; t < 16; ++t)
      if (sb * 16 + t < n)
        G[(long)(row0 + sb * 16 + t) * g.kq() + c] = off + z[t];
  }
}

// A tile held transposed, [column][64 tokens] float32: the 16-byte blocks of
// a column are permuted by the column, so that stores with lanes along the
// columns' quads and reads of one block of 16 columns both spread over the
// banks.
__device__ __forceinline__ int tr_at(int col, int blk) {
  return col * CH + ((blk ^ ((col >> 2) & 15) ^ ((col & 3) << 2)) << 2);
}
__device__ __forceinline__ f32x8 tr_ld8(const float* tile, int col, int t) {
  const f32x4 a = *(const f32x4*)(tile + tr_at(col, t >> 2));
  const f32x4 b = *(const f32x4*)(tile + tr_at(col, (t >> 2) + 1));
  return f32x8{a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
}

// 4 consecutive elements of a row; with vec their place is 8- or 16-byte
// aligned. Elements from ``lim`` on are zero.
template <typename T>
__device__ __forceinline__ f32x4 ld4(const T* p, int lim, int vec) {
  f32x4 v = {0.f, 0.f, 0.f, 0.f};
  if (vec) {
    if (lim > 0) {
      T t[4];
      __builtin_memcpy(t, __builtin_assume_aligned(p, 4 * sizeof(T)),
                       sizeof(t));
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = El<T>::ld(t[j]);
    }
  } else {
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j < lim) v[j] = El<T>::ld(p[j]);
  }
  return v;
}

// Values of columns e0 .. e0+NE-1, transposed, zero past the chunk and past
// vdim. A thread turns 4 tokens x 4 columns.
template <typename T, int NE>
__device__ __forceinline__ void stage_vt(float* vt, const T* __restrict__ proj,
                                         long ps, const Gla& g, int h, int row0,
                                         int n, int e0, int vec) {
  constexpr int Q = NE / 4;
  constexpr int NU = (Q * 16 + 255) / 256;
  f32x4 x[NU][4];
#pragma unroll
  for (int u = 0; u < NU; ++u) {
    const int i = threadIdx.x + u * 256;
    const int e = i % Q * 4, t = i / Q * 4;
    const int lim = i < Q * 16 ? g.vdim - e0 - e : 0;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      x[u][j] = ld4<T>(proj + (long)(row0 + min(t + j, n - 1)) * ps +
                           g.v_off() + h * g.vdim + e0 + e,
                       t + j < n ? lim : 0, vec);
  }
#pragma unroll
  for (int u = 0; u < NU; ++u) {
    const int i = threadIdx.x + u * 256;
    const int e = i % Q * 4, t = i / Q * 4;
    if (i < Q * 16)
#pragma unroll
      for (int c = 0; c < 4; ++c)
        *(f32x4*)(vt + tr_at(e + c, t >> 2)) =
            f32x4{x[u][0][c], x[u][1][c], x[u][2][c], x[u][3][c]};
  }
}

// U[chunk][h][e][d] = sum_s v_s[e] k_s[d] exp(G_end[d] - G_s[d]).
// grid (chunks, heads, ceil(vdim / 64)); wave w owns 16 value rows.
template <typename T, int DT>              // DT = ceil(dim / 16), rounded up
__global__ void __launch_bounds__(256)
k_gla_state(float* __restrict__ U, const float* __restrict__ G,
            const T* __restrict__ proj, long ps,
            const int* __restrict__ chunks, Gla g, int vec) {
  extern __shared__ __align__(16) char smem[];
  float* kt = (float*)smem;                // [DT * 16][CH], see tr_at
  float* vt = kt + DT * 16 * CH;           // [64][CH]
  const int row0 = chunks[blockIdx.x * 3 + 1], n = chunks[blockIdx.x * 3 + 2];
  const int h = blockIdx.y, e0 = blockIdx.z * 64;
  const float* gend = G + (long)(row0 + n - 1) * g.kq() + h * g.dim;
  constexpr int Q = DT * 4;                // quads of channels
  constexpr int NU = (Q * 16 + 255) / 256;
#pragma unroll
  for (int u = 0; u < NU; ++u) {
    const int i = threadIdx.x + u * 256;
    const int d = i % Q * 4, t = i / Q * 4;
    const int lim = i < Q * 16 ? g.dim - d : 0;
    const f32x4 ge = ld4<float>(gend + d, lim, vec);
    f32x4 k[4], gg[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const long row = row0 + min(t + j, n - 1);
      k[j] = ld4<T>(proj + row * ps + g.k_off() + h * g.dim + d,
                    t + j < n ? lim : 0, vec);
      gg[j] = ld4<float>(G + row * g.kq() + h * g.dim + d, lim, vec);
    }
    if (i < Q * 16)
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        f32x4 v;
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] = k[j][c] * El<T>::ex(ge[c] - gg[j][c]);
        *(f32x4*)(kt + tr_at(d + c, t >> 2)) = v;
      }
  }
  stage_vt<T, 64>(vt, proj, ps, g, h, row0, n, e0, vec);
  __syncthreads();
  const int w = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int l15 = lane & 15, lg = lane >> 4;
  if (e0 + w * 16 >= g.vdim) return;
  f32x8 a[2];
#pragma unroll
  for (int k = 0; k < 2; ++k)
    a[k] = tr_ld8(vt, w * 16 + l15, k * 32 + 8 * lg);
  float* u = U + ((long)blockIdx.x * g.heads + h) * g.vdim * g.dim;
#pragma unroll
  for (int dt = 0; dt < DT; ++dt) {
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < 2; ++k)
      acc = mma(a[k], tr_ld8(kt, dt * 16 + l15, k * 32 + 8 * lg), acc);
    const int d = dt * 16 + l15;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int e = e0 + w * 16 + 4 * lg + r;
      if (e < g.vdim && d < g.dim) u[(long)e * g.dim + d] = acc[r];
    }
  }
}

// U becomes the start state of each chunk; the last state goes to the slot.
// spans [P][4]: first chunk, chunks, first position, sequence. grid
// (state values / 256, P); NB chunks are read ahead of the recurrence.
__global__ void __launch_bounds__(256)
k_gla_scan(float* __restrict__ U, const float* __restrict__ G,
           float* __restrict__ states, const int* __restrict__ chunks,
           const int* __restrict__ spans, const int* __restrict__ slots,
           Gla g) {
  constexpr int NB = 8;
  const long size = (long)g.heads * g.vdim * g.dim;
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= size) return;
  const int* sp = spans + blockIdx.y * 4;
  const int c0 = sp[0], nc = sp[1];
  float* slot = states + (long)slots[sp[3]] * size + i;
  const int hd = (int)(i / ((long)g.vdim * g.dim)) * g.dim + (int)(i % g.dim);
  float s = sp[2] == 0 ? 0.f : *slot;
  for (int c = 0; c < nc; c += NB) {
    float u[NB], e[NB];
#pragma unroll
    for (int j = 0; j < NB; ++j)
      if (c + j < nc) {
        const int* ck = chunks + (c0 + c + j) * 3;
        u[j] = U[(long)(c0 + c + j) * size + i];
        e[j] = G[(long)(ck[1] + ck[2] - 1) * g.kq() + hd];
      }
#pragma unroll
    for (int j = 0; j < NB; ++j)
      if (c + j < nc) {
        U[(long)(c0 + c + j) * size + i] = s;
        s = fmaf(expf(e[j]), s, u[j]);
      }
  }
  *slot = s;
}

// A[chunk][h][CH][CH], zero above the diagonal. grid (chunks, heads); wave w
// owns query rows 16w .. 16w+15. Channels go by slices of 64.
template <typename T>
__global__ void __launch_bounds__(256)
k_gla_scores(float* __restrict__ A, const float* __restrict__ G,
             const T* __restrict__ proj, long ps,
             const int* __restrict__ chunks, Gla g, int vec) {
  constexpr int DS = 64 + 4;
  __shared__ __align__(16) float qs[CH * DS], ks[CH * DS], gs[CH * DS];
  const int row0 = chunks[blockIdx.x * 3 + 1], n = chunks[blockIdx.x * 3 + 2];
  const int h = blockIdx.y;
  const int w = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int l15 = lane & 15, lg = lane >> 4;
  const float scale = 1.f / sqrtf((float)g.dim);
  f32x4 off[3];
#pragma unroll
  for (int j = 0; j < 3; ++j) off[j] = f32x4{0.f, 0.f, 0.f, 0.f};
  float diag[4] = {0.f, 0.f, 0.f, 0.f};    // rows t = l15, columns 4 lg + r

  for (int d0 = 0; d0 < g.dim; d0 += 64) {
    __syncthreads();
    {
      f32x4 q[4], k[4], gg[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int i = threadIdx.x + u * 256;
        const int t = i >> 4, d = d0 + (i & 15) * 4;
        // past the chunk: G of the last token, so that no exponent is positive
        const long row = row0 + min(t, n - 1);
        const int lim = g.dim - d, on = t < n ? lim : 0;
        q[u] = ld4<T>(proj + row * ps + h * g.dim + d, on, vec);
        k[u] = ld4<T>(proj + row * ps + g.k_off() + h * g.dim + d, on, vec);
        gg[u] = ld4<float>(G + row * g.kq() + h * g.dim + d, lim, vec);
      }
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int i = threadIdx.x + u * 256;
        const int at = (i >> 4) * DS + (i & 15) * 4;
        *(f32x4*)(qs + at) = q[u] * scale;
        *(f32x4*)(ks + at) = k[u];
        *(f32x4*)(gs + at) = gg[u];
      }
    }
    __syncthreads();
    if (w > 0) {
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const int c = k * 32 + 8 * lg;
        const f32x8 ref = ld8(gs + (w * 16 - 1) * DS + c);
        f32x8 a = ld8(qs + (w * 16 + l15) * DS + c);
        const f32x8 ga = ld8(gs + (w * 16 + l15) * DS + c);
#pragma unroll
        for (int j = 0; j < 8; ++j) a[j] *= El<T>::ex(ga[j] - ref[j]);
#pragma unroll
        for (int jb = 0; jb < 3; ++jb)
          if (jb < w) {
            f32x8 b = ld8(ks + (jb * 16 + l15) * DS + c);
            const f32x8 gb = ld8(gs + (jb * 16 + l15) * DS + c);
#pragma unroll
            for (int j = 0; j < 8; ++j) b[j] *= El<T>::ex(ref[j] - gb[j]);
            off[jb] = mma(a, b, off[jb]);
          }
      }
    }
    const float* qr = qs + (w * 16 + l15) * DS;
    const float* gr = gs + (w * 16 + l15) * DS;
    for (int d = 0; d < 64 && d0 + d < g.dim; d += 4) {
      const f32x4 q4 = *(const f32x4*)(qr + d), gt = *(const f32x4*)(gr + d);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int s = w * 16 + 4 * lg + r;
        const f32x4 k4 = *(const f32x4*)(ks + s * DS + d);
        const f32x4 g4 = *(const f32x4*)(gs + s * DS + d);
#pragma unroll
        for (int j = 0; j < 4; ++j)        // s > t is dropped below
          diag[r] = fmaf(q4[j] * k4[j], El<T>::ex(fminf(gt[j] - g4[j], 0.f)),
                         diag[r]);
      }
    }
  }
  float* a = A + ((long)blockIdx.x * g.heads + h) * CH * CH;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
#pragma unroll
    for (int jb = 0; jb < 3; ++jb)
      if (jb < w) a[(w * 16 + 4 * lg + r) * CH + jb * 16 + l15] = off[jb][r];
    const int s = 4 * lg + r;
    a[(w * 16 + l15) * CH + w * 16 + s] = s <= l15 ? diag[r] : 0.f;
    for (int jb = w + 1; jb < 4; ++jb)
      a[(w * 16 + 4 * lg + r) * CH + jb * 16 + l15] = 0.f;
  }
}

// o = (q exp(G)) S + A V, head norm, gate. grid (chunks, heads); wave w owns
// 16 tokens and all of vdim, which goes by tiles of 32 columns held in LDS.
// DK = ceil(dim / 32), NV = ceil(vdim / 32), both rounded up.
template <typename T, int DK, int NV>
__global__ void __launch_bounds__(256)
k_gla_out(T* __restrict__ out, long os, const float* __restrict__ S,
          const float* __restrict__ A, const float* __restrict__ G,
          const T* __restrict__ proj, long ps, const float* __restrict__ nw,
          const int* __restrict__ chunks, Gla g, float eps, int vec) {
  constexpr int DS = DK * 32 + 4;
  __shared__ __align__(16) float st[32 * DS];
  __shared__ __align__(16) float vt[32 * CH];
  const int row0 = chunks[blockIdx.x * 3 + 1], n = chunks[blockIdx.x * 3 + 2];
  const int h = blockIdx.y;
  const int w = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int l15 = lane & 15, lg = lane >> 4;
  const float scale = 1.f / sqrtf((float)g.dim);
  const float* s0 = S + ((long)blockIdx.x * g.heads + h) * g.vdim * g.dim;

  f32x8 aq[DK], aa[2];
  const int t = w * 16 + l15;
#pragma unroll
  for (int k = 0; k < DK; ++k) {
    const long row = row0 + min(t, n - 1);
    const int d = k * 32 + 8 * lg;
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      const int lim = t < n ? g.dim - d - 4 * b : 0;
      const f32x4 q = ld4<T>(proj + row * ps + h * g.dim + d + 4 * b, lim, vec);
      const f32x4 gg = ld4<float>(G + row * g.kq() + h * g.dim + d + 4 * b, lim,
                                  vec);
#pragma unroll
      for (int j = 0; j < 4; ++j) aq[k][4 * b + j] = q[j] * scale * El<T>::ex(gg[j]);
    }
  }
#pragma unroll
  for (int k = 0; k < 2; ++k)
    aa[k] = ld8(A + (((long)blockIdx.x * g.heads + h) * CH + t) * CH + k * 32 +
                8 * lg);

  f32x4 o[NV * 2];
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int e0 = v * 32;
    if (e0 < g.vdim) {                     // uniform
      __syncthreads();
      f32x4 x[DK];
#pragma unroll
      for (int u = 0; u < DK; ++u) {
        const int i = threadIdx.x + u * 256;
        const int e = i / (DK * 8), d = i % (DK * 8) * 4;
        x[u] = ld4<float>(s0 + (long)(e0 + e) * g.dim + d,
                          e0 + e < g.vdim ? g.dim - d : 0, vec);
      }
#pragma unroll
      for (int u = 0; u < DK; ++u) {
        const int i = threadIdx.x + u * 256;
        *(f32x4*)(st + i / (DK * 8) * DS + i % (DK * 8) * 4) = x[u];
      }
      stage_vt<T, 32>(vt, proj, ps, g, h, row0, n, e0, vec);
      __syncthreads();
#pragma unroll
      for (int c = 0; c < 2; ++c) {
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < DK; ++k)
          acc = mma(aq[k], ld8(st + (c * 16 + l15) * DS + k * 32 + 8 * lg), acc);
#pragma unroll
        for (int k = 0; k < 2; ++k)
          acc = mma(aa[k], tr_ld8(vt, c * 16 + l15, k * 32 + 8 * lg), acc);
        o[v * 2 + c] = acc;
      }
    } else {
      o[v * 2] = o[v * 2 + 1] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    float ss = 0.f;                        // columns past vdim are zero
#pragma unroll
    for (int c = 0; c < NV * 2; ++c) ss = fmaf(o[c][r], o[c][r], ss);
    ss = row16_sum(ss);
    const int tr = w * 16 + 4 * lg + r;
    if (tr >= n) continue;
    const float inv = 1.f / sqrtf(ss / (float)g.vdim + eps);
    const T* gate = proj + (long)(row0 + tr) * ps + g.g_off() + h * g.vdim;
    T* dst = out + (long)(row0 + tr) * os + h * g.vdim;
#pragma unroll
    for (int c = 0; c < NV * 2; ++c) {
      const int e = c * 16 + l15;
      if (e < g.vdim) {
        const float gv = El<T>::ld(gate[e]);
        dst[e] = El<T>::st(o[c][r] * inv * nw[e] * gv * sigmoid_f(gv));
      }
    }
  }
}

// One token per sequence: S <- S diag(alpha) + v k^T, o = S q (float32, to
// ``o`` [B][H vdim]). grid (heads, ceil(vdim / 16), B), 4 value rows a wave.
// lpr: lanes that share a value row, a power of two; with vec each takes 4
// channels at a time, otherwise one.
template <typename T>
__global__ void __launch_bounds__(256)
k_gla_decode(float* __restrict__ o, float* __restrict__ states,
             const T* __restrict__ proj, long ps, const float* __restrict__ a2,
             const float* __restrict__ bias, const int* __restrict__ pos,
             const int* __restrict__ slots, Gla g, int lpr, int vec) {
  __shared__ __align__(16) float q[256], k[256], al[256], a1[256];
  const int h = blockIdx.x, b = blockIdx.z, tid = threadIdx.x;
  const T* pr = proj + (long)b * ps;
  const bool fresh = pos[b] == 0;
  if (tid < g.rank) a1[tid] = El<T>::ld(pr[g.a_off() + tid]);
  __syncthreads();
  if (tid < g.dim) {
    const int c = h * g.dim + tid;
    float z = bias[c];
    for (int r = 0; r < g.rank; ++r) z = fmaf(a2[(long)c * g.rank + r], a1[r], z);
    al[tid] = expf(log_decay(z, 1.f / g.tau));
    q[tid] = El<T>::ld(pr[c]) / sqrtf((float)g.dim);
    k[tid] = El<T>::ld(pr[g.k_off() + c]);
  }
  __syncthreads();
  const int w = tid >> 6, lane = tid & 63;
  const int rpw = 64 / lpr, sub = lane % lpr, rw = lane / lpr;
  float* base = states +
      ((long)slots[b] * g.heads + h) * g.vdim * g.dim;
  for (int i = 0; i < 4; i += rpw) {
    const int e = blockIdx.y * 16 + w * 4 + i + rw;
    const bool on = i + rw < 4 && e < g.vdim;
    float acc = 0.f;
    if (on) {
      float* s = base + (long)e * g.dim;
      const float v = El<T>::ld(pr[g.v_off() + h * g.vdim + e]);
      if (vec) {
        for (int d = sub * 4; d < g.dim; d += lpr * 4) {
          f32x4 x = fresh ? f32x4{0.f, 0.f, 0.f, 0.f} : *(f32x4*)(s + d);
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            x[j] = fmaf(al[d + j], x[j], v * k[d + j]);
            acc = fmaf(x[j], q[d + j], acc);
          }
          *(f32x4*)(s + d) = x;
        }
      } else {
        for (int d = sub; d < g.dim; d += lpr) {
          const float x = fmaf(al[d], fresh ? 0.f : s[d], v * k[d]);
          acc = fmaf(x, q[d], acc);
          s[d] = x;
        }
      }
    }
    for (int off = lpr >> 1; off; off >>= 1) acc += __shfl_xor(acc, off);
    if (on && sub == 0) o[(long)b * g.vo() + h * g.vdim + e] = acc;
  }
}

// out = rms(o) * nw * silu(gate) per head. grid (heads, B), one wave.
template <typename T>
__global__ void __launch_bounds__(64)
k_gla_gate_out(T* __restrict__ out, long os, const float* __restrict__ o,
               const T* __restrict__ proj, long ps,
               const float* __restrict__ nw, Gla g, float eps) {
  const int h = blockIdx.x, b = blockIdx.y;
  const float* x = o + (long)b * g.vo() + h * g.vdim;
  float ss = 0.f;
  for (int e = threadIdx.x; e < g.vdim; e += 64) ss = fmaf(x[e], x[e], ss);
  ss = wave_reduce_sum(ss);
  const float inv = 1.f / sqrtf(ss / (float)g.vdim + eps);
  for (int e = threadIdx.x; e < g.vdim; e += 64) {
    const float gv = El<T>::ld(proj[(long)b * ps + g.g_off() + h * g.vdim + e]);
    out[(long)b * os + h * g.vdim + e] =
        El<T>::st(x[e] * inv * nw[e] * gv * sigmoid_f(gv));
  }
}

template <typename T>
void run_gla_decode(T* out, long os, float* o, float* states, const T* proj,
                    long ps, const float* a2, const float* bias,
                    const float* nw, const int* pos, const int* slots, int B,
                    Gla g, float eps, hipStream_t stream) {
  const int vec = g.dim % 4 == 0;
  const int need = vec ? g.dim / 4 : g.dim;
  int lpr = 16;
  while (lpr < 64 && lpr < need) lpr <<= 1;
  hipLaunchKernelGGL(k_gla_decode<T>, dim3(g.heads, (g.vdim + 15) / 16, B),
                     dim3(256), 0, stream, o, states, proj, ps, a2, bias, pos,
                     slots, g, lpr, vec);
  hipLaunchKernelGGL(k_gla_gate_out<T>, dim3(g.heads, B), dim3(64), 0, stream,
                     out, os, o, proj, ps, nw, g, eps);
}

template <typename T, int DT>
void launch_state(float* U, const float* G, const T* proj, long ps,
                  const int* chunks, int n, Gla g, int vec,
                  hipStream_t stream) {
  const size_t lds = 4 * (DT * 16 + 64) * CH;
  static bool set = false;
  if (!set) {
    (void)hipFuncSetAttribute((const void*)k_gla_state<T, DT>,
                              hipFuncAttributeMaxDynamicSharedMemorySize,
                              160 * 1024);
    set = true;
  }
  hipLaunchKernelGGL((k_gla_state<T, DT>),
                     dim3(n, g.heads, (g.vdim + 63) / 64), dim3(256), lds,
                     stream, U, G, proj, ps, chunks, g, vec);
}

template <typename T>
void run_gla_prefill(T* out, long os, const T* proj, long ps, const float* a2,
                     const float* bias, const float* nw, float* states,
                     const int* chunks, int n, const int* spans, int P,
                     const int* slots, float* G, float* U, float* A, Gla g,
                     float eps, hipStream_t stream) {
  hipLaunchKernelGGL(k_gla_gate<T>, dim3(n, (g.kq() + 63) / 64), dim3(256),
                     4 * CH * g.rank, stream, G, proj, ps, a2, bias, chunks, g);
  // quads of q, k, v, G and S lie on 8- and 16-byte borders
  const int vec = g.dim % 4 == 0 && g.vdim % 4 == 0 && ps % 4 == 0 &&
                  (size_t)proj % 16 == 0;
  const int dt = (g.dim + 15) / 16;
  if (dt <= 2) launch_state<T, 2>(U, G, proj, ps, chunks, n, g, vec, stream);
  else if (dt <= 4) launch_state<T, 4>(U, G, proj, ps, chunks, n, g, vec, stream);
  else if (dt <= 8) launch_state<T, 8>(U, G, proj, ps, chunks, n, g, vec, stream);
  else launch_state<T, 16>(U, G, proj, ps, chunks, n, g, vec, stream);
  const long size = (long)g.heads * g.vdim * g.dim;
  hipLaunchKernelGGL(k_gla_scan, dim3((size + 255) / 256, P), dim3(256), 0,
                     stream, U, G, states, chunks, spans, slots, g);
  hipLaunchKernelGGL(k_gla_scores<T>, dim3(n, g.heads), dim3(256), 0, stream,
                     A, G, proj, ps, chunks, g, vec);
  const dim3 go(n, g.heads);
#define OUT(DK, NV)                                                         \
  hipLaunchKernelGGL((k_gla_out<T, DK, NV>), go, dim3(256), 0, stream, out, \
                     os, U, A, G, proj, ps, nw, chunks, g, eps, vec)
#define BY_NV(DK)                           \
  do {                                      \
    if (g.vdim <= 64) OUT(DK, 2);           \
    else if (g.vdim <= 128) OUT(DK, 4);     \
    else if (g.vdim <= 256) OUT(DK, 8);     \
    else OUT(DK, 16);                       \
  } while (0)
  if (g.dim <= 32) BY_NV(1);
  else if (g.dim <= 64) BY_NV(2);
  else if (g.dim <= 128) BY_NV(4);
  else BY_NV(8);
#undef BY_NV
#undef OUT
}

}  // namespace

extern "C" {

void fei_gla_decode(void* out, long os, float* o, float* states,
                    const void* proj, long ps, const float* a2,
                    const float* bias, const float* nw, const int* pos,
                    const int* slots, int B, int heads, int dim, int vdim,
                    int rank, float tau, float eps, int f32,
                    hipStream_t stream) {
  const Gla g{heads, dim, vdim, rank, tau};
  if (f32)
    run_gla_decode<float>((float*)out, os, o, states, (const float*)proj, ps,
                          a2, bias, nw, pos, slots, B, g, eps, stream);
  else
    run_gla_decode<u16>((u16*)out, os, o, states, (const u16*)proj, ps, a2,
                        bias, nw, pos, slots, B, g, eps, stream);
}

// Workspaces: G [T][H dim], U [chunks][H][vdim][dim], A [chunks][H][64][64].
void fei_gla_prefill(void* out, long os, const void* proj, long ps,
                     const float* a2, const float* bias, const float* nw,
                     float* states, const int* chunks, int n_chunks,
                     const int* spans, int n_spans, const int* slots, float* G,
                     float* U, float* A, int heads, int dim, int vdim,
                     int rank, float tau, float eps, int f32,
                     hipStream_t stream) {
  const Gla g{heads, dim, vdim, rank, tau};
  if (f32)
    run_gla_prefill<float>((float*)out, os, (const float*)proj, ps, a2, bias,
                           nw, states, chunks, n_chunks, spans, n_spans, slots,
                           G, U, A, g, eps, stream);
  else
    run_gla_prefill<u16>((u16*)out, os, (const u16*)proj, ps, a2, bias, nw,
                         states, chunks, n_chunks, spans, n_spans, slots, G, U,
                         A, g, eps, stream);
}

}  // extern "C"
