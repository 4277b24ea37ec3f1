// Latent attention (keys and values are linear maps of a cached latent c, and
// all heads share one rotated key part) with a sliding window, over a paged
// cache of rows [c (kv_rank) | rotated key (rot)].
//
// Decode attends in the latent space: with q' = W_uk^T q per head, a score is
// q' . c + q_rot . k_rot, so all heads read the same rows (k_latent_decode,
// one MFMA tile of 16 heads), and W_uv is applied to the weighted latent
// (k_latent_out). Prompts expand the latents to per-head keys and values with
// one matrix product and run a flash kernel over them (k_window_prefill),
// which costs fewer operations per key when many queries share it.
//
// T is u16 (bfloat16 bits) or float. Scores, weights and sums are float32;
// where a weight enters a bfloat16 matrix product it is given as a high and a
// low part, so that it keeps about 16 bits.
#include "fei_attn.h"
#include "fei_common.h"
#include "fei_mma.h"

namespace {

constexpr float NEG_INF = -__builtin_inff();

struct Geo {           // sizes of one mixer
  int heads, dim, rot, vdim, kr;
  float scale;
  int window;          // keys a query sees, itself included; 0 = all
};

// Norm of the latent and rotation of the shared key part of one token, into
// its cache row. ``ckr`` points at the row's kr + rot projected values.
template <typename T>
__device__ __forceinline__ void append_row(const T* __restrict__ ckr,
                                           T* __restrict__ dst,
                                           const float* __restrict__ nw,
                                           const float* __restrict__ cs,
                                           int kr, int rot, float eps,
                                           float* red) {
  float ss = 0.f;
  for (int i = threadIdx.x; i < kr; i += blockDim.x) {
    const float v = El<T>::ld(ckr[i]);
    ss = fmaf(v, v, ss);
  }
  ss = block_reduce_sum(ss, red);
  const float inv = 1.f / sqrtf(ss / (float)kr + eps);
  for (int i = threadIdx.x; i < kr; i += blockDim.x)
    dst[i] = El<T>::st(El<T>::ld(ckr[i]) * inv * nw[i]);
  for (int i = threadIdx.x; i < rot / 2; i += blockDim.x) {
    const float u = El<T>::ld(ckr[kr + 2 * i]);
    const float v = El<T>::ld(ckr[kr + 2 * i + 1]);
    const float c = cs[2 * i], s = cs[2 * i + 1];
    dst[kr + 2 * i] = El<T>::st(u * c - v * s);
    dst[kr + 2 * i + 1] = El<T>::st(v * c + u * s);
  }
}

// Prompt rows: cache row, and the rotated part of every query in place.
template <typename T>
__global__ void __launch_bounds__(256)
k_latent_append(T* __restrict__ proj, long ps, T* __restrict__ rows,
                const float* __restrict__ nw, const float* __restrict__ rotab,
                const int* __restrict__ pos, const int* __restrict__ row_seq,
                const int* __restrict__ table, int W, int bs_log, Geo g,
                float eps) {
  __shared__ float red[4];
  const int t = blockIdx.x;
  const int p = pos[t];
  T* pr = proj + (long)t * ps;
  const float* cs = rotab + (long)p * g.rot;
  const int D = g.dim + g.rot;
  append_row<T>(pr + (long)g.heads * D,
                rows + cache_row(table, W, row_seq[t], p, bs_log) *
                           (g.kr + g.rot),
                nw, cs, g.kr, g.rot, eps, red);
  const int half = g.rot / 2;
  for (int i = threadIdx.x; i < g.heads * half; i += blockDim.x) {
    const int h = i / half, j = i - h * half;
    T* q = pr + (long)h * D + g.dim + 2 * j;
    const float u = El<T>::ld(q[0]), v = El<T>::ld(q[1]);
    const float c = cs[2 * j], s = cs[2 * j + 1];
    q[0] = El<T>::st(u * c - v * s);
    q[1] = El<T>::st(v * c + u * s);
  }
}

// Decode rows: grid (heads + 1, ceil(kr / 128), B). Block x = heads appends
// the token's cache row; the others make 128 columns of q' = W_uk^T q of one
// head (16 groups of 8 columns x 16 groups of rows of W_uk), and block y = 0
// the rotated query.
template <typename T, bool VEC>
__global__ void __launch_bounds__(256)
k_latent_absorb(const T* __restrict__ proj, long ps, T* __restrict__ qa,
                const T* __restrict__ wuk, T* __restrict__ rows,
                const float* __restrict__ nw, const float* __restrict__ rotab,
                const int* __restrict__ pos, const int* __restrict__ table,
                int W, int bs_log, Geo g, float eps) {
  __shared__ float qs[256];
  __shared__ float part[16][128];
  const int h = blockIdx.x, b = blockIdx.z, tid = threadIdx.x;
  const int p = pos[b];
  const int D = g.dim + g.rot, R = g.kr + g.rot;
  const T* pr = proj + (long)b * ps;
  const float* cs = rotab + (long)p * g.rot;
  if (h == g.heads) {
    if (blockIdx.y == 0)
      append_row<T>(pr + (long)g.heads * D,
                    rows + cache_row(table, W, b, p, bs_log) * R, nw, cs,
                    g.kr, g.rot, eps, qs);
    return;
  }
  const T* q = pr + (long)h * D;
  T* qo = qa + ((long)b * g.heads + h) * R;
  for (int i = tid; i < g.dim; i += 256) qs[i] = El<T>::ld(q[i]);
  if (blockIdx.y == 0) {
    for (int i = tid; i < g.rot / 2; i += 256) {
      const float u = El<T>::ld(q[g.dim + 2 * i]);
      const float v = El<T>::ld(q[g.dim + 2 * i + 1]);
      const float c = cs[2 * i], s = cs[2 * i + 1];
      qo[g.kr + 2 * i] = El<T>::st(u * c - v * s);
      qo[g.kr + 2 * i + 1] = El<T>::st(v * c + u * s);
    }
  }
  __syncthreads();
  const int cg = tid & 15, dg = tid >> 4;
  const int col = blockIdx.y * 128 + cg * 8;
  float acc[8];
#pragma unroll
  for (int j = 0; j < 8; ++j) acc[j] = 0.f;
  if (col < g.kr) {
    const T* w = wuk + (long)h * g.dim * g.kr + col;
    if (VEC) {
#pragma unroll 4
      for (int d = dg; d < g.dim; d += 16) {
        const auto wv = ld8(w + (long)d * g.kr);
        const float qd = qs[d];
#pragma unroll
        for (int j = 0; j < 8; ++j) acc[j] = fmaf(qd, get8(wv, j), acc[j]);
      }
    } else {
      for (int d = dg; d < g.dim; d += 16)
#pragma unroll
        for (int j = 0; j < 8; ++j)
          if (col + j < g.kr)
            acc[j] = fmaf(qs[d], El<T>::ld(w[(long)d * g.kr + j]), acc[j]);
    }
  }
#pragma unroll
  for (int j = 0; j < 8; ++j) part[dg][cg * 8 + j] = acc[j];
  __syncthreads();
  const int c = blockIdx.y * 128 + tid;
  if (tid < 128 && c < g.kr) {
    float v = 0.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) v += part[i][tid];
    qo[c] = El<T>::st(v);
  }
}

// Decode partials. grid (splits, ceil(heads / 16 NH), B). The visible
// keys of row b are cut into ``splits`` chunks of a multiple of KT keys; a
// block walks its chunk in tiles of KT cached rows held in LDS, which NH groups
// of 4 waves use for 16 heads each. For the scores a group's waves share out
// the 32-wide steps along a row (their sums meet in LDS), for the weighted sum
// the columns.
// NCT: 16-column tiles of the latent per wave (kr <= 64 * NCT).
// part_o [B, H, splits, kr] unnormalised, part_ml [B, H, splits, 2].
template <typename T, int NCT, int NH>
__global__ void __launch_bounds__(256 * NH)
k_latent_decode(const T* __restrict__ qa, const T* __restrict__ rows,
                float* __restrict__ part_o, float* __restrict__ part_ml,
                const int* __restrict__ pos, const int* __restrict__ table,
                int W, int bs_log, Geo g, int splits, int KT, int Rs,
                int vec) {
  typedef typename El<T>::frag frag;
  constexpr int NP = Parts<T>::n;
  constexpr int NQ = 9;                    // steps per wave: R <= 4 * 9 * 32
  constexpr int NT = 256 * NH;
  constexpr int NL = 9;                    // row loads in flight per thread
  extern __shared__ __align__(16) char smem[];
  const int R = g.kr + g.rot;
  const int KP = (KT + 31) / 32 * 32;      // P columns, zero beyond KT
  const int KPs = KP + 8;
  T* ks = (T*)smem;                        // [KP][Rs]
  const int split = blockIdx.x, b = blockIdx.z;
  const int tid = threadIdx.x, grp = tid >> 8, w = (tid >> 6) & 3;
  const int lane = tid & 63;
  const int h0 = (blockIdx.y * NH + grp) * 16;
  // per group: [NP][16][KPs], [4][16][KT + 1], [16]
  T* ph = ks + KP * Rs + grp * NP * 16 * KPs;
  float* ss = (float*)(ks + KP * Rs + NH * NP * 16 * KPs) +
              grp * (64 * (KT + 1) + 16);
  float* al = ss + 64 * (KT + 1);
  const int l15 = lane & 15, lg = lane >> 4;
  const int p = pos[b];
  const int k0 = first_key(p, g.window);
  const int n = p + 1 - k0;
  const int chunk = ((n + splits - 1) / splits + KT - 1) / KT * KT;
  const int lo = split * chunk, hi = min(lo + chunk, n);
  const int nh = min(16, g.heads - h0);    // may be 0 or less in a last group

  if (lo >= hi) {
    const int h = tid & 255;
    if (h < nh) {
      float* ml = part_ml + (((long)b * g.heads + h0 + h) * splits + split) * 2;
      ml[0] = NEG_INF;
      ml[1] = 0.f;
    }
    return;
  }

  // queries of this wave's steps, zero beyond the heads and beyond R
  const int ksteps = (R + 31) / 32;
  frag q[NQ];
  {
    const T* qr = qa + ((long)b * g.heads + h0 + max(min(l15, nh - 1), 0)) * R;
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
      const int k = w + 4 * i;
#pragma unroll
      for (int j = 0; j < 8; ++j) q[i][j] = 0;
      if (k < ksteps && l15 < nh) {
        const int c = k * 32 + 8 * lg;
        if (vec) {
          if (c < R) q[i] = ld8(qr + c);
        } else {
#pragma unroll
          for (int j = 0; j < 8; ++j)
            if (c + j < R) q[i][j] = qr[c + j];
        }
      }
    }
  }
  for (int i = tid & 255; i < NP * 16 * KPs; i += 256) ph[i] = El<T>::st(0.f);
  for (int i = KT * Rs + tid; i < KP * Rs; i += NT) ks[i] = El<T>::st(0.f);

  f32x4 acc[NCT];
#pragma unroll
  for (int i = 0; i < NCT; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  // row 4w + lg of the scores is this 16-lane group's
  float m = NEG_INF, l = 0.f;

  for (int t0 = lo; t0 < hi; t0 += KT) {
    __syncthreads();
    if (vec) {
      const int nv = Rs / 8 - 1;           // vec8 slots that may be read
      // i / nv for i < 2^16, as a product (nv > 1)
      const unsigned per = 0xffffffffu / (unsigned)nv + 1u;
      for (int i0 = tid; i0 < KT * nv; i0 += NT * NL) {
        frag v[NL];
#pragma unroll
        for (int u = 0; u < NL; ++u) {
          const int i = i0 + u * NT;
          const int r = __umulhi((unsigned)i, per), c = (i - r * nv) * 8;
#pragma unroll
          for (int j = 0; j < 8; ++j) v[u][j] = 0;
          if (i < KT * nv && t0 + r < hi && c < R)
            v[u] = ld8(rows +
                       cache_row(table, W, b, k0 + t0 + r, bs_log) * R + c);
        }
#pragma unroll
        for (int u = 0; u < NL; ++u) {
          const int i = i0 + u * NT;
          const int r = __umulhi((unsigned)i, per), c = (i - r * nv) * 8;
          if (i < KT * nv) st8(ks + r * Rs + c, v[u]);
        }
      }
    } else {
      for (int i = tid; i < KT * Rs; i += NT) {
        const int r = i / Rs, c = i - r * Rs;
        ks[i] = (t0 + r < hi && c < R)
                    ? rows[cache_row(table, W, b, k0 + t0 + r, bs_log) * R + c]
                    : El<T>::st(0.f);
      }
    }
    __syncthreads();
    for (int kt = 0; kt < KT / 16; ++kt) {
      f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < NQ; ++i)
        if (w + 4 * i < ksteps)
          s = mma(q[i], ld8(ks + (kt * 16 + l15) * Rs + (w + 4 * i) * 32 +
                            8 * lg), s);
#pragma unroll
      for (int r = 0; r < 4; ++r)
        ss[(w * 16 + 4 * lg + r) * (KT + 1) + kt * 16 + l15] = s[r];
    }
    __syncthreads();
    {
      const int row = 4 * w + lg;
      float sv[4];
      float mx = m;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int c = l15 + 16 * i;
        sv[i] = NEG_INF;
        if (c < KT && t0 + c < hi) {
          const float* x = ss + row * (KT + 1) + c;
          const int st = 16 * (KT + 1);
          sv[i] = ((x[0] + x[st]) + (x[2 * st] + x[3 * st])) * g.scale;
        }
        mx = fmaxf(mx, sv[i]);
      }
      mx = row16_max(mx);
      const float a = El<T>::ex(m - mx);   // a tile has a visible key: mx is finite
      float sum = 0.f;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int c = l15 + 16 * i;
        if (c < KT) {
          const float e = El<T>::ex(sv[i] - mx);
          sum += e;
#pragma unroll
          for (int pi = 0; pi < NP; ++pi)
            ph[(pi * 16 + row) * KPs + c] = part_of<T>(e, pi);
        }
      }
      l = l * a + row16_sum(sum);
      m = mx;
      if (l15 == 0) al[row] = a;
    }
    __syncthreads();
    float a[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) a[r] = al[4 * lg + r];
#pragma unroll
    for (int i = 0; i < NCT; ++i) {
      const int c0 = (w + 4 * i) * 16;
      if (c0 < g.kr) {
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[i][r] *= a[r];
        for (int k = 0; k < KP / 32; ++k) {
          frag bv;
#pragma unroll
          for (int j = 0; j < 8; ++j)
            bv[j] = ks[(k * 32 + 8 * lg + j) * Rs + c0 + l15];
#pragma unroll
          for (int i2 = 0; i2 < NP; ++i2)
            acc[i] = mma(ld8(ph + (i2 * 16 + l15) * KPs + k * 32 + 8 * lg), bv,
                         acc[i]);
        }
      }
    }
  }

  const int row = 4 * w + lg;
  if (l15 == 0 && row < nh) {
    float* ml = part_ml + (((long)b * g.heads + h0 + row) * splits + split) * 2;
    ml[0] = m;
    ml[1] = l;
  }
#pragma unroll
  for (int i = 0; i < NCT; ++i) {
    const int c = (w + 4 * i) * 16 + l15;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int h = 4 * lg + r;
      if (h < nh && c < g.kr)
        part_o[(((long)b * g.heads + h0 + h) * splits + split) * g.kr + c] =
            acc[i][r];
    }
  }
}

// Combine the partials of one head, apply W_uv and the gate. grid (heads,
// ceil(vdim / 16), B); a wave takes 4 value rows, whose first weights it reads
// ahead of the combination.
template <typename T, bool VEC>
__global__ void __launch_bounds__(256)
k_latent_out(T* __restrict__ out, long os, const float* __restrict__ part_o,
             const float* __restrict__ part_ml, const T* __restrict__ wuv,
             const T* __restrict__ gate, long gs, Geo g, int splits) {
  __shared__ float wt[64];
  __shared__ __align__(16) float o[1024];
  const int h = blockIdx.x, b = blockIdx.z, tid = threadIdx.x;
  const int w = tid >> 6, lane = tid & 63;
  const long bh = (long)b * g.heads + h;
  const int v0 = blockIdx.y * 16 + w * 4;
  const T* wr = wuv + ((long)h * g.vdim + v0) * g.kr;
  typename El<T>::frag pre[4];
  if (VEC) {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (v0 + i < g.vdim && lane * 8 < g.kr)
        pre[i] = ld8(wr + (long)i * g.kr + lane * 8);
  }
  if (tid < 64) {
    const bool on = tid < splits;
    const float m = on ? part_ml[(bh * splits + tid) * 2] : NEG_INF;
    const float l = on ? part_ml[(bh * splits + tid) * 2 + 1] : 0.f;
    const float mx = wave_reduce_max(m);
    const float e = l > 0.f ? El<T>::ex(m - mx) : 0.f;
    const float sum = wave_reduce_sum(e * l);
    wt[tid] = e / sum;
  }
  __syncthreads();
  for (int c = tid; c < g.kr; c += 256) {
    const float* po = part_o + bh * splits * g.kr + c;
    float v = 0.f;
    int s = 0;
    for (; s + 8 <= splits; s += 8) {
      float x[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) x[u] = po[(long)(s + u) * g.kr];
#pragma unroll
      for (int u = 0; u < 8; ++u)          // an empty split wrote nothing
        v = wt[s + u] > 0.f ? fmaf(wt[s + u], x[u], v) : v;
    }
    for (; s < splits; ++s)
      v = wt[s] > 0.f ? fmaf(wt[s], po[(long)s * g.kr], v) : v;
    o[c] = v;
  }
  __syncthreads();
  float acc[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    if (v0 + i >= g.vdim) continue;
    const T* r = wr + (long)i * g.kr;
    if (VEC) {
      for (int c = lane * 8; c < g.kr; c += 512) {
        const auto wv = c == lane * 8 ? pre[i] : ld8(r + c);
#pragma unroll
        for (int j = 0; j < 8; ++j) acc[i] = fmaf(o[c + j], get8(wv, j), acc[i]);
      }
    } else {
      for (int c = lane; c < g.kr; c += 64)
        acc[i] = fmaf(o[c], El<T>::ld(r[c]), acc[i]);
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const float v = wave_reduce_sum(acc[i]);
    if (lane == 0 && v0 + i < g.vdim) {
      const int col = h * g.vdim + v0 + i;
      out[(long)b * os + col] = El<T>::st(
          v * sigmoid_f(El<T>::ld(gate[(long)b * gs + col])));
    }
  }
}

// Cached rows of the keys that the prompt portions see, packed one portion
// after another: latents [n, kr] and rotated parts [n, rot].
// spans [P][5]: first row, rows, first position, first key, first packed key.
template <typename T>
__global__ void __launch_bounds__(128)
k_latent_gather(T* __restrict__ c, T* __restrict__ kr_out,
                const T* __restrict__ rows, const int* __restrict__ owner,
                const int* __restrict__ spans, const int* __restrict__ table,
                int W, int bs_log, int seq0, Geo g, int vec) {
  const int i = blockIdx.x;
  const int p = owner[i];
  const int key = spans[p * 5 + 3] + i - spans[p * 5 + 4];
  const int R = g.kr + g.rot;
  const T* src = rows + cache_row(table, W, seq0 + p, key, bs_log) * R;
  if (vec) {
    for (int j = threadIdx.x * 8; j < g.kr; j += blockDim.x * 8)
      st8(c + (long)i * g.kr + j, ld8(src + j));
    for (int j = threadIdx.x * 8; j < g.rot; j += blockDim.x * 8)
      st8(kr_out + (long)i * g.rot + j, ld8(src + g.kr + j));
  } else {
    for (int j = threadIdx.x; j < g.kr; j += blockDim.x)
      c[(long)i * g.kr + j] = src[j];
    for (int j = threadIdx.x; j < g.rot; j += blockDim.x)
      kr_out[(long)i * g.rot + j] = src[g.kr + j];
  }
}

// Flash attention of prompt portions over expanded keys and values.
// grid (heads, query tiles), NW waves; a wave owns 16 query rows, and the
// block walks the keys they see in tiles of 64 held in LDS: keys row-major,
// values transposed. tiles [.][2]: portion, first row in it (a tile of the
// plan is 128 rows; with 4 waves two blocks share it, blockIdx.z).
// KS = ceil((dim + rot) / 32), DC = ceil(vdim / 16), rounded up to what is
// instantiated; queries are zero beyond dim + rot, columns beyond vdim are
// not stored.
template <typename T, int KS, int DC, int NW>
__global__ void __launch_bounds__(NW * 64, 2)
k_window_prefill(T* __restrict__ out, long os, const T* __restrict__ proj,
                 long ps, const T* __restrict__ kv, const T* __restrict__ krot,
                 const int* __restrict__ spans, const int* __restrict__ tiles,
                 int gate_off, Geo g, int vec) {
  typedef typename El<T>::frag frag;
  constexpr int NP = Parts<T>::n;
  constexpr int NT = NW * 64;
  constexpr int DS = KS * 32 + 8;          // odd count of 16-byte slots
  constexpr int PS = 64 + 8;
  extern __shared__ __align__(16) char smem[];
  T* kt = (T*)smem;                        // [64][DS]
  T* vt = kt + 64 * DS;                    // [DC * 16][64], see vt_at
  T* pl = vt + DC * 16 * 64;               // [NW][NP][16][PS]

  // heads run fastest, so that with 8 | heads a head stays on one XCD and
  // neighbouring tiles find their common keys in its L2
  const int h = blockIdx.x;
  const int* sp = spans + tiles[blockIdx.y * 2] * 5;
  const int row0 = sp[0], cnt = sp[1], pos0 = sp[2], key0 = sp[3], at0 = sp[4];
  const int q0 = tiles[blockIdx.y * 2 + 1] + blockIdx.z * NW * 16;
  if (q0 >= cnt) return;
  const int qn = min(16 * NW, cnt - q0);
  const int tid = threadIdx.x, w = tid >> 6, lane = tid & 63;
  const int l15 = lane & 15, lg = lane >> 4;
  const int D = g.dim + g.rot;
  const long kvs = (long)g.heads * (g.dim + g.vdim);
  const T* kh = kv + (long)h * g.dim;
  const T* vh = kv + (long)g.heads * g.dim + (long)h * g.vdim;

  frag aq[KS];
  {
    const int r = min(w * 16 + l15, qn - 1);
    const T* q = proj + (long)(row0 + q0 + r) * ps + (long)h * D;
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      const int c = k * 32 + 8 * lg;
#pragma unroll
      for (int j = 0; j < 8; ++j) aq[k][j] = 0;
      if (vec) {
        if (c < D) aq[k] = ld8(q + c);
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j)
          if (c + j < D) aq[k][j] = q[c + j];
      }
    }
  }
  float m[4], l[4];
  f32x4 o[DC];
#pragma unroll
  for (int r = 0; r < 4; ++r) { m[r] = NEG_INF; l[r] = 0.f; }
#pragma unroll
  for (int d = 0; d < DC; ++d) o[d] = f32x4{0.f, 0.f, 0.f, 0.f};

  // positions of this tile's queries and of the keys any of them sees
  const int qa = pos0 + q0, qb = qa + qn - 1;
  const int klo = max(first_key(qa, g.window), key0) & ~63;
  // this wave's own range: tiles outside it are staged for the others only
  const int wa = qa + w * 16, wb = min(wa + 15, qb);
  const int wlo = first_key(wa, g.window);
  T* pw = pl + w * NP * 16 * PS;
  const float scale = g.scale * El<T>::base;

  for (int t0 = klo; t0 <= qb; t0 += 64) {
    __syncthreads();
    if (vec) {
      // all loads before the first store. Keys outside the range and columns
      // past the head's sizes read some valid place: the queries are zero
      // there, the scores masked, the output columns dropped.
      constexpr int NV = KS * 4, NC = DC * 2;
      constexpr int UK = (64 * NV + NT - 1) / NT, UV = (32 * NC + NT - 1) / NT;
      frag kf[UK], va[UV], vb[UV];
#pragma unroll
      for (int u = 0; u < UK; ++u) {
        const int i = tid + u * NT;
        const int r = i / NV, c = (i - r * NV) * 8;
        const int n = at0 + min(max(t0 + r, key0), qb) - key0;
        const T* src = c >= g.dim && c < D
                           ? krot + (long)n * g.rot + c - g.dim
                           : kh + (long)n * kvs + (c < g.dim ? c : 0);
        kf[u] = ld8(src);
      }
#pragma unroll
      for (int u = 0; u < UV; ++u) {
        const int i = tid + u * NT;
        const int r = i / NC * 2, c = min(i % NC * 8, g.vdim - 8);
        const int ka = min(max(t0 + r, key0), qb) - key0;
        const int kb = min(max(t0 + r + 1, key0), qb) - key0;
        va[u] = ld8(vh + (long)(at0 + ka) * kvs + c);
        vb[u] = ld8(vh + (long)(at0 + kb) * kvs + c);
      }
#pragma unroll
      for (int u = 0; u < UK; ++u) {
        const int i = tid + u * NT;
        const int r = i / NV, c = (i - r * NV) * 8;
        if (64 * NV % NT == 0 || i < 64 * NV) st8(kt + r * DS + c, kf[u]);
      }
#pragma unroll
      for (int u = 0; u < UV; ++u) {
        const int i = tid + u * NT;
        const int r = i / NC * 2, c = i % NC * 8;
        if (32 * NC % NT == 0 || i < 32 * NC)
#pragma unroll
          for (int j = 0; j < 8; ++j) {
            T two[2] = {(T)va[u][j], (T)vb[u][j]};
            __builtin_memcpy(vt + vt_at(c + j, r), two, sizeof(two));
          }
      }
    } else {
      for (int i = tid; i < 64 * KS * 32; i += NT) {
        const int r = i / (KS * 32), c = i - r * (KS * 32);
        const int key = t0 + r;
        T v = El<T>::st(0.f);
        if (key >= key0 && key <= qb && c < D) {
          const long n = at0 + key - key0;
          v = c < g.dim ? kh[n * kvs + c] : krot[n * g.rot + c - g.dim];
        }
        kt[r * DS + c] = v;
      }
      for (int i = tid; i < 64 * DC * 16; i += NT) {
        const int r = i / (DC * 16), c = i - r * (DC * 16);
        const int key = t0 + r;
        T v = El<T>::st(0.f);
        if (key >= key0 && key <= qb && c < g.vdim)
          v = vh[(long)(at0 + key - key0) * kvs + c];
        vt[vt_at(c, r)] = v;
      }
    }
    __syncthreads();
    if (t0 > wb || t0 + 63 < wlo) continue;

    f32x4 s[4];
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      s[c] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < KS; ++k)
        s[c] = mma(aq[k], ld8(kt + (c * 16 + l15) * DS + k * 32 + 8 * lg), s[c]);
    }
    // no mask where every query of the wave sees every key of the tile
    const bool edge = t0 + 63 > wa || t0 < key0 ||
                      (g.window > 0 && wb - t0 >= g.window);
    float al[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int qp = wa + 4 * lg + r;
      float mx = m[r];
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        float v = s[c][r] * scale;
        if (edge) {
          const int key = t0 + c * 16 + l15;
          if (key > qp || key < key0 || (g.window > 0 && qp - key >= g.window))
            v = NEG_INF;
        }
        s[c][r] = v;
        mx = fmaxf(mx, v);
      }
      mx = row16_max(mx);
      const bool any = mx > NEG_INF;       // no key so far: keep zeros
      al[r] = any ? El<T>::exb(m[r] - mx) : 1.f;
      m[r] = mx;
      float sum = 0.f;                     // of this lane's columns
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        const float e = any ? El<T>::exb(s[c][r] - mx) : 0.f;
        sum += e;
#pragma unroll
        for (int pi = 0; pi < NP; ++pi)
          pw[(pi * 16 + 4 * lg + r) * PS + c * 16 + l15] = part_of<T>(e, pi);
      }
      l[r] = fmaf(l[r], al[r], sum);
    }
    // pw belongs to this wave alone: its LDS operations stay in order
    __builtin_amdgcn_wave_barrier();
    frag ap[NP][2];
#pragma unroll
    for (int pi = 0; pi < NP; ++pi)
#pragma unroll
      for (int k = 0; k < 2; ++k)
        ap[pi][k] = ld8(pw + (pi * 16 + l15) * PS + k * 32 + 8 * lg);
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int d = 0; d < DC; ++d) {
#pragma unroll
      for (int r = 0; r < 4; ++r) o[d][r] *= al[r];
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const frag bv = ld8(vt + vt_at(d * 16 + l15, k * 32 + 8 * lg));
#pragma unroll
        for (int pi = 0; pi < NP; ++pi) o[d] = mma(ap[pi][k], bv, o[d]);
      }
    }
  }

  float lsum[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) lsum[r] = row16_sum(l[r]);
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int q = w * 16 + 4 * lg + r;
    if (q >= qn) continue;
    const float inv = 1.f / lsum[r];       // a query always sees itself
    const T* gate = proj + (long)(row0 + q0 + q) * ps + gate_off +
                    (long)h * g.vdim;
    T* dst = out + (long)(row0 + q0 + q) * os + (long)h * g.vdim;
#pragma unroll
    for (int d = 0; d < DC; ++d) {
      const int c = d * 16 + l15;
      if (c < g.vdim)
        dst[c] = El<T>::st(o[d][r] * inv * sigmoid_f(El<T>::ld(gate[c])));
    }
  }
}

template <typename T>
int run_decode(T* out, long os, const T* proj, long ps, const T* wuk,
               const T* wuv, const float* nw, const float* rotab, T* rows,
               const int* pos, const int* table, T* qa, float* part_o,
               float* part_ml, int B, int W, int bs_log, Geo g, float eps,
               int splits, int tile, hipStream_t stream) {
  const int R = g.kr + g.rot;
  const bool vkr = g.kr % 8 == 0;
  const dim3 ga(g.heads + 1, (g.kr + 127) / 128, B);
  if (vkr)
    hipLaunchKernelGGL((k_latent_absorb<T, true>), ga, dim3(256), 0, stream,
                       proj, ps, qa, wuk, rows, nw, rotab, pos, table, W,
                       bs_log, g, eps);
  else
    hipLaunchKernelGGL((k_latent_absorb<T, false>), ga, dim3(256), 0, stream,
                       proj, ps, qa, wuk, rows, nw, rotab, pos, table, W,
                       bs_log, g, eps);

  const int Rs = (R + 31) / 32 * 32 + 8;
  const int nh = g.heads > 16 ? 2 : 1;     // groups of 16 heads per block
  auto lds = [&](int KT) {
    const int KP = (KT + 31) / 32 * 32;
    return (size_t)sizeof(T) * (KP * Rs + nh * Parts<T>::n * 16 * (KP + 8)) +
           4 * nh * (64 * (KT + 1) + 16);
  };
  int KT = tile;
  while (KT > 16 && lds(KT) > 160 * 1024) KT >>= 1;
  if (lds(KT) > 160 * 1024 || R > 1152) return 1;
  const dim3 gd(splits, (g.heads + 16 * nh - 1) / (16 * nh), B);
#define DEC(N, H)                                                            \
  do {                                                                       \
    static bool set = false;                                                 \
    if (!set) {                                                              \
      (void)hipFuncSetAttribute((const void*)k_latent_decode<T, N, H>,       \
                                hipFuncAttributeMaxDynamicSharedMemorySize,  \
                                160 * 1024);                                 \
      set = true;                                                            \
    }                                                                        \
    hipLaunchKernelGGL((k_latent_decode<T, N, H>), gd, dim3(256 * H),        \
                       lds(KT), stream, qa, rows, part_o, part_ml, pos,      \
                       table, W, bs_log, g, splits, KT, Rs, R % 8 == 0);     \
  } while (0)
#define BY_NCT(H)               \
  do {                          \
    if (nct <= 2) DEC(2, H);    \
    else if (nct <= 4) DEC(4, H); \
    else if (nct <= 8) DEC(8, H); \
    else DEC(16, H);            \
  } while (0)
  const int nct = (g.kr + 63) / 64;
  if (nh == 2) BY_NCT(2); else BY_NCT(1);
#undef BY_NCT
#undef DEC

  const dim3 go(g.heads, (g.vdim + 15) / 16, B);
  const T* gate = proj + (long)g.heads * (g.dim + g.rot) + R;
  if (vkr)
    hipLaunchKernelGGL((k_latent_out<T, true>), go, dim3(256), 0, stream, out,
                       os, part_o, part_ml, wuv, gate, ps, g, splits);
  else
    hipLaunchKernelGGL((k_latent_out<T, false>), go, dim3(256), 0, stream,
                       out, os, part_o, part_ml, wuv, gate, ps, g, splits);
  return 0;
}

template <typename T, int KS, int DC>
void launch_window(T* out, long os, const T* proj, long ps, const T* kv,
                   const T* krot, const int* spans, const int* tiles,
                   int n_tiles, Geo g, int vec, hipStream_t stream) {
  constexpr int NW = sizeof(T) == 2 ? 8 : 4;
  const size_t lds = sizeof(T) * (64 * (KS * 32 + 8) + DC * 16 * 64 +
                                  NW * Parts<T>::n * 16 * 72);
  static bool set = false;
  if (!set) {
    (void)hipFuncSetAttribute((const void*)k_window_prefill<T, KS, DC, NW>,
                              hipFuncAttributeMaxDynamicSharedMemorySize,
                              160 * 1024);
    set = true;
  }
  const dim3 grid(g.heads, n_tiles, NW == 8 ? 1 : 2);
  const int gate_off = g.heads * (g.dim + g.rot) + g.kr + g.rot;
  hipLaunchKernelGGL((k_window_prefill<T, KS, DC, NW>), grid, dim3(NW * 64), lds,
                     stream, out, os, proj, ps, kv, krot, spans, tiles,
                     gate_off, g, vec);
}

template <typename T>
void run_window(T* out, long os, const T* proj, long ps, const T* kv,
                const T* krot, const int* spans, const int* tiles,
                int n_tiles, Geo g, hipStream_t stream) {
  const int vec = g.dim % 8 == 0 && g.rot % 8 == 0 && g.vdim % 8 == 0 &&
                  ps % 8 == 0;
  const int ks = (g.dim + g.rot + 31) / 32, dc = (g.vdim + 15) / 16;
#define WIN(KS, DC) launch_window<T, KS, DC>(out, os, proj, ps, kv, krot,    \
                                             spans, tiles, n_tiles, g, vec,  \
                                             stream)
#define BY_DC(KS)                        \
  do {                                   \
    if (dc <= 4) WIN(KS, 4);             \
    else if (dc <= 8) WIN(KS, 8);        \
    else WIN(KS, 16);                    \
  } while (0)
  if (ks <= 2) BY_DC(2);
  else if (ks <= 4) BY_DC(4);
  else if (ks <= 6) BY_DC(6);
  else BY_DC(8);
#undef BY_DC
#undef WIN
}

}  // namespace

extern "C" {

// tile: keys per LDS tile, 16, 32 or 64; fewer are taken if they do not fit.
// Returns 0, or 1 if the sizes do not fit the kernel's LDS tiles.
int fei_latent_decode(void* out, long os, const void* proj, long ps,
                      const void* wuk, const void* wuv, const float* nw,
                      const float* rotab, void* rows, const int* pos,
                      const int* table, void* qa, float* part_o,
                      float* part_ml, int B, int W, int bs_log, int heads,
                      int dim, int rot, int vdim, int kr, float scale,
                      int window, float eps, int splits, int tile, int f32,
                      hipStream_t stream) {
  const Geo g{heads, dim, rot, vdim, kr, scale, window};
  if (f32)
    return run_decode<float>((float*)out, os, (const float*)proj, ps,
                             (const float*)wuk, (const float*)wuv, nw, rotab,
                             (float*)rows, pos, table, (float*)qa, part_o,
                             part_ml, B, W, bs_log, g, eps, splits, tile, stream);
  return run_decode<u16>((u16*)out, os, (const u16*)proj, ps,
                         (const u16*)wuk, (const u16*)wuv, nw, rotab,
                         (u16*)rows, pos, table, (u16*)qa, part_o, part_ml, B,
                         W, bs_log, g, eps, splits, tile, stream);
}

void fei_latent_append(void* proj, long ps, void* rows, const float* nw,
                       const float* rotab, const int* pos, const int* row_seq,
                       const int* table, int T, int W, int bs_log, int heads,
                       int dim, int rot, int vdim, int kr, float eps, int f32,
                       hipStream_t stream) {
  const Geo g{heads, dim, rot, vdim, kr, 1.f, 0};
  if (f32)
    hipLaunchKernelGGL(k_latent_append<float>, dim3(T), dim3(256), 0, stream,
                       (float*)proj, ps, (float*)rows, nw, rotab, pos,
                       row_seq, table, W, bs_log, g, eps);
  else
    hipLaunchKernelGGL(k_latent_append<u16>, dim3(T), dim3(256), 0, stream,
                       (u16*)proj, ps, (u16*)rows, nw, rotab, pos, row_seq,
                       table, W, bs_log, g, eps);
}

void fei_latent_gather(void* c, void* krot, const void* rows,
                       const int* owner, const int* spans, const int* table,
                       int n, int W, int bs_log, int seq0, int kr, int rot,
                       int f32, hipStream_t stream) {
  const Geo g{0, 0, rot, 0, kr, 1.f, 0};
  const int vec = kr % 8 == 0 && rot % 8 == 0;
  if (f32)
    hipLaunchKernelGGL(k_latent_gather<float>, dim3(n), dim3(128), 0, stream,
                       (float*)c, (float*)krot, (const float*)rows, owner,
                       spans, table, W, bs_log, seq0, g, vec);
  else
    hipLaunchKernelGGL(k_latent_gather<u16>, dim3(n), dim3(128), 0, stream,
                       (u16*)c, (u16*)krot, (const u16*)rows, owner, spans,
                       table, W, bs_log, seq0, g, vec);
}

void fei_window_prefill(void* out, long os, const void* proj, long ps,
                        const void* kv, const void* krot, const int* spans,
                        const int* tiles, int n_tiles, int heads, int dim,
                        int rot, int vdim, int kr, float scale, int window,
                        int f32, hipStream_t stream) {
  const Geo g{heads, dim, rot, vdim, kr, scale, window};
  if (f32)
    run_window<float>((float*)out, os, (const float*)proj, ps,
                      (const float*)kv, (const float*)krot, spans, tiles,
                      n_tiles, g, stream);
  else
    run_window<u16>((u16*)out, os, (const u16*)proj, ps, (const u16*)kv,
                    (const u16*)krot, spans, tiles, n_tiles, g, stream);
}

}  // extern "C"
