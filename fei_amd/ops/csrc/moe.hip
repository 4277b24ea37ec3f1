// Mixture of experts: sigmoid router, experts W_down relu(W_up h)^2.
//
// Few rows: k_moe_up_gemv chooses the experts and makes the activations of
// the chosen ones, k_moe_out_gemv their weighted sum, the mixer's output
// product and the residual sum. More rows: k_moe_route chooses, k_moe_plan
// sorts (row, choice) pairs by expert into slots and cuts them into tiles of
// one expert each, grouped matrix products run over the tiles, and k_moe_add
// gathers each row's results. Nothing depends on host values: a grid is
// launched for the largest possible number of tiles.
//
// T is u16 (bfloat16 bits) or float.
#include "fei_common.h"
#include "fei_epilogue.h"
#include "fei_mma.h"

namespace {

constexpr int MAX_E = 1024;

// Place of expert e among all, largest logit first, the lower index on ties.
// z in LDS.
__device__ __forceinline__ int rank_of(const float* z, int E, int e) {
  const float v = z[e];
  int r = 0;
  for (int i = 0; i < E; ++i) r += z[i] > v || (z[i] == v && i < e);
  return r;
}

// Choice of one row by a block (or wave) of ``nt`` threads: ids and weights
// of its ``top`` experts. z: E floats of LDS, filled and visible.
// total: sum of the chosen scores; the caller reduces and scales.
__device__ __forceinline__ float choose(const float* z, int E, int top,
                                        int tid, int nt, int* ids, float* w) {
  float mine = 0.f;
  for (int e = tid; e < E; e += nt) {
    const int r = rank_of(z, E, e);
    if (r < top) {
      const float s = sigmoid_f(z[e]);
      ids[r] = e;
      w[r] = s;
      mine += s;
    }
  }
  return mine;
}

// One wave per row.
__global__ void __launch_bounds__(256)
k_moe_route(int* __restrict__ ids, float* __restrict__ w,
            const float* __restrict__ logits, int T, int E, int top,
            float scale) {
  __shared__ float zs[4][MAX_E];
  const int wid = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int t = blockIdx.x * 4 + wid;
  const bool on = t < T;
  float* z = zs[wid];
  if (on) {
    for (int e = lane; e < E; e += 64) z[e] = logits[(long)t * E + e];
    // a choice that no logit takes (not a number) is still some expert
    for (int k = lane; k < top; k += 64) {
      ids[(long)t * top + k] = k;
      w[(long)t * top + k] = 0.f;
    }
  }
  __syncthreads();
  float sum = 0.f;
  if (on)
    sum = choose(z, E, top, lane, 64, ids + (long)t * top,
                 w + (long)t * top);
  sum = wave_reduce_sum(sum) + 1e-20f;
  __syncthreads();
  if (on)
    for (int k = lane; k < top; k += 64) {
      const float s = w[(long)t * top + k];
      w[(long)t * top + k] = s / sum * scale;
    }
}

// Slots sorted by expert: order[slot] = row, place[row * top + k] = slot;
// tiles [.][3]: expert, first slot, slots (at most ``rows``); count[0] tiles.
// One block.
__global__ void __launch_bounds__(1024)
k_moe_plan(int* __restrict__ order, int* __restrict__ place,
           int* __restrict__ tiles, int* __restrict__ count,
           const int* __restrict__ ids, int n, int E, int top, int rows,
           int max_tiles) {
  __shared__ int cnt[MAX_E], slots[MAX_E], first[MAX_E];
  const int tid = threadIdx.x;
  cnt[tid] = 0;
  __syncthreads();
  for (int i = tid; i < n; i += 1024) atomicAdd(&cnt[ids[i]], 1);
  __syncthreads();
  const int c = cnt[tid], nt = (c + rows - 1) / rows;
  slots[tid] = c;
  first[tid] = nt;
  __syncthreads();
  for (int d = 1; d < MAX_E; d <<= 1) {    // inclusive sums
    const int a = tid >= d ? slots[tid - d] : 0;
    const int b = tid >= d ? first[tid - d] : 0;
    __syncthreads();
    slots[tid] += a;
    first[tid] += b;
    __syncthreads();
  }
  const int s0 = slots[tid] - c, t0 = first[tid] - nt;
  if (tid == MAX_E - 1) count[0] = min(first[tid], max_tiles);
  for (int k = 0; k < nt; ++k)
    if (t0 + k < max_tiles) {
      int* t = tiles + (t0 + k) * 3;
      t[0] = tid;
      t[1] = s0 + k * rows;
      t[2] = min(rows, c - k * rows);
    }
  cnt[tid] = s0;                           // next free slot
  __syncthreads();
  for (int i = tid; i < n; i += 1024) {
    const int s = atomicAdd(&cnt[ids[i]], 1);
    order[s] = i / top;
    place[i] = s;
  }
}

// Grouped product of any sizes: out[slot, n] = w[expert][n] . x[row], with
// row = order[slot] or the slot itself; ACT: relu(.)^2. grid (ceil(N / 64),
// tiles of 32 slots); a wave makes 16 columns of all slots.
template <typename T, bool VEC>
__global__ void __launch_bounds__(256)
k_moe_gemm(T* __restrict__ out, const T* __restrict__ x,
           const T* __restrict__ w, const int* __restrict__ order,
           const int* __restrict__ tiles, const int* __restrict__ count,
           int N, int K, int act) {
  typedef typename El<T>::frag frag;
  constexpr int BK = 64, S = BK + 8;
  __shared__ __align__(16) T xs[32 * S], ws[64 * S];
  if ((int)blockIdx.y >= count[0]) return;
  const int* t = tiles + blockIdx.y * 3;
  const int s0 = t[1], cnt = t[2], n0 = blockIdx.x * 64;
  const T* we = w + (long)t[0] * N * K;
  const int tid = threadIdx.x, wid = tid >> 6, lane = tid & 63;
  const int l15 = lane & 15, lg = lane >> 4;
  // 8 columns of a row a thread: one row of x, two of w
  const int r = tid >> 3, c = (tid & 7) * 8;
  const int slot = s0 + min(r, cnt - 1);
  const T* xr = x + (long)(order ? order[slot] : slot) * K;
  const T* w0 = we + (long)min(n0 + r, N - 1) * K;
  const T* w1 = we + (long)min(n0 + r + 32, N - 1) * K;
  auto get = [&](const T* p, int k) {
    frag v;
    if (VEC) {
      if (k + c < K) return ld8(p + k + c);
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] = 0;
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] = k + c + j < K ? p[k + c + j] : (T)0;
    }
    return v;
  };
  f32x4 acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
  frag fx = get(xr, 0), fa = get(w0, 0), fb = get(w1, 0);
  for (int k0 = 0; k0 < K; k0 += BK) {
    __syncthreads();
    st8(xs + r * S + c, fx);
    st8(ws + r * S + c, fa);
    st8(ws + (r + 32) * S + c, fb);
    __syncthreads();
    if (k0 + BK < K) {
      fx = get(xr, k0 + BK);
      fa = get(w0, k0 + BK);
      fb = get(w1, k0 + BK);
    }
#pragma unroll
    for (int k = 0; k < BK / 32; ++k) {
      const frag a = ld8(ws + (wid * 16 + l15) * S + k * 32 + 8 * lg);
#pragma unroll
      for (int i = 0; i < 2; ++i)
        acc[i] = mma(a, ld8(xs + (i * 16 + l15) * S + k * 32 + 8 * lg),
                     acc[i]);
    }
  }
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    if (i * 16 + l15 >= cnt) continue;
    T* dst = out + (long)(s0 + i * 16 + l15) * N;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int n = n0 + wid * 16 + 4 * lg + j;
      if (n < N) dst[n] = El<T>::st(act ? relu2(acc[i][j]) : acc[i][j]);
    }
  }
}

// 64 lanes x 16 bytes from memory straight into LDS, lane i at lds + 16 i
// (a byte address, the same in all lanes).
__device__ __forceinline__ void load_lds(const u16* src, u32 lds) {
  u32 keep;
  asm volatile(
      "s_mov_b32 %0, m0\n\t"
      "s_mov_b32 m0, %2\n\t"
      "s_nop 0\n\t"
      "global_load_lds_dwordx4 %1, off\n\t"
      "s_mov_b32 m0, %0"
      : "=&s"(keep)
      : "v"(src), "s"(lds)
      : "memory");
}

// The same for bfloat16 with K % 64 == 0 and N % 4 == 0: tiles of 128 slots x
// 32 WI columns, 4 waves of 64 slots x 16 WI columns, S LDS buffers of 64
// steps of K filled by direct loads. The 16-byte places of a row are permuted
// by the row (in the address that a lane reads, since LDS is filled in lane
// order), so that the fragment reads of 16 rows spread over the banks.
// An XCD gets consecutive blocks, in groups of 8 tiles of slots times all nx of
// columns, slots first: its L2 then holds their common rows and weights.
template <int WI, int S>
__global__ void __launch_bounds__(256, 2)
k_moe_gemm_big(u16* __restrict__ out, const u16* __restrict__ x,
               const u16* __restrict__ w, const int* __restrict__ order,
               const int* __restrict__ tiles, const int* __restrict__ count,
               int nx, int N, int K, int act) {
  constexpr int TN = 32 * WI;
  constexpr int BUF = (128 + TN) * 64;     // elements: 128 rows of x, TN of w
  constexpr int LOADS = 4 + WI;            // a wave's per buffer: x, w
  extern __shared__ __align__(16) u16 buf[];
  const int total = count[0] * nx, per = (total + 7) / 8;
  const int id = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
  if ((int)(blockIdx.x >> 3) >= per || id >= total) return;
  const int g0 = id / (8 * nx) * 8, gm = min(8, count[0] - g0);
  const int gr = id - g0 * nx;
  const int* t = tiles + (g0 + gr % gm) * 3;
  const int s0 = t[1], cnt = t[2], n0 = gr / gm * TN;
  const u16* we = w + (long)t[0] * N * K;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l15 = lane & 15, lg = lane >> 4;
  // 8 rows a load; the place of a row's 8 values depends on the row
  const int r8 = lane >> 3, c8 = ((lane & 7) ^ r8) * 8;
  const u16* src[LOADS];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int slot = s0 + min((wid * 4 + i) * 8 + r8, cnt - 1);
    src[i] = x + (long)(order ? order[slot] : slot) * K + c8;
  }
#pragma unroll
  for (int i = 0; i < WI; ++i)
    src[4 + i] = we + (long)min(n0 + (wid * WI + i) * 8 + r8, N - 1) * K + c8;
  const u32 lds = (u32)(uintptr_t)(__attribute__((address_space(3))) u16*)buf;
  const int steps = K / 64;
  // past the end the last steps are read again, into a buffer that is free
  auto load = [&](int step, int b, int i) {
    load_lds(src[i] + min(step, steps - 1) * 64,
             lds + b * BUF * 2 +
                 (i < 4 ? (wid * 4 + i) * 1024
                        : 16384 + (wid * WI + i - 4) * 1024));
  };
  const int xm = (wid & 1) * 64, wm = (wid >> 1) * 16 * WI;
  struct Frags {
    s16x8 w[WI], x[4];
  };
  auto read = [&](Frags& f, int b, int kk, int i) {
    const int c = ((kk * 4 + lg) ^ (l15 & 7)) * 8;
    const u16* bx = buf + b * BUF;
    if (i < 4) f.x[i] = ld8(bx + (xm + i * 16 + l15) * 64 + c);
    f.w[i] = ld8(bx + (128 + wm + i * 16 + l15) * 64 + c);
  };
  f32x4 acc[WI][4];
#pragma unroll
  for (int i = 0; i < WI; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int s = 0; s < S; ++s)
#pragma unroll
    for (int i = 0; i < LOADS; ++i) load(s, s, i);
  asm volatile("s_waitcnt vmcnt(%0)\n\ts_barrier" ::"n"((S - 1) * LOADS)
               : "memory");
  Frags f0, f1;
#pragma unroll
  for (int i = 0; i < WI; ++i) read(f0, 0, 0, i);
  int b = 0;                               // buffer of step k
  // Fragments of 32 steps of K are read ahead of the products with the 32
  // before. At the barrier all waves have the second half of buffer b, which
  // can be filled again, and the loads of the next one have arrived. Reads
  // and loads go out between the matrix instructions.
  for (int k = 0; k < steps; ++k) {
#pragma unroll
    for (int i = 0; i < WI; ++i) {
      read(f1, b, 1, i);
#pragma unroll
      for (int j = 0; j < 4; ++j)
        acc[i][j] = mma(f0.w[i], f0.x[j], acc[i][j]);
      __builtin_amdgcn_sched_barrier(0);
    }
    asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)\n\ts_barrier" ::"n"(
                     (S - 2) * LOADS)
                 : "memory");
    const int nb = b == S - 1 ? 0 : b + 1;
#pragma unroll
    for (int i = 0; i < WI; ++i) {
      read(f0, nb, 0, i);
      load(k + S, b, i);
      if (WI + i < LOADS) load(k + S, b, WI + i);
#pragma unroll
      for (int j = 0; j < 4; ++j)
        acc[i][j] = mma(f1.w[i], f1.x[j], acc[i][j]);
      __builtin_amdgcn_sched_barrier(0);
    }
    b = nb;
  }
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int r = xm + j * 16 + l15;
    if (r >= cnt) continue;
    u16* dst = out + (long)(s0 + r) * N;
#pragma unroll
    for (int i = 0; i < WI; ++i) {
      const int n = n0 + wm + i * 16 + 4 * lg;
      if (n >= N) continue;
      u16 v[4];
#pragma unroll
      for (int e = 0; e < 4; ++e)
        v[e] = El<u16>::st(act ? relu2(acc[i][j][e]) : acc[i][j][e]);
      __builtin_memcpy(dst + n, v, sizeof(v));
    }
  }
}

template <int WI, int S>
void launch_big(u16* out, const u16* x, const u16* w, const int* order,
                const int* tiles, const int* count, int max_tiles, int N,
                int K, int act, hipStream_t stream) {
  constexpr int lds = S * (128 + 32 * WI) * 64 * 2;
  static bool set = false;
  if (!set) {
    (void)hipFuncSetAttribute((const void*)k_moe_gemm_big<WI, S>,
                              hipFuncAttributeMaxDynamicSharedMemorySize,
                              lds);
    set = true;
  }
  const int nx = (N + 32 * WI - 1) / (32 * WI);
  hipLaunchKernelGGL((k_moe_gemm_big<WI, S>),
                     dim3((nx * max_tiles + 7) / 8 * 8), dim3(256), lds,
                     stream, out, x, w, order, tiles, count, nx, N, K, act);
}

// x[t] += mult * sum_k w[t, k] y[place[t, k]]. One block per row.
template <typename T>
__global__ void __launch_bounds__(256)
k_moe_add(float* __restrict__ x, const T* __restrict__ y,
          const int* __restrict__ place, const float* __restrict__ w, int C,
          int top, float mult, int vec) {
  const long t = blockIdx.x;
  const int* pl = place + t * top;
  const float* wt = w + t * top;
  float* xr = x + t * C;
  if (vec) {
    for (int c = threadIdx.x * 8; c < C; c += 2048) {
      float a[8];
#pragma unroll
      for (int j = 0; j < 8; ++j) a[j] = 0.f;
      for (int k = 0; k < top; ++k) {
        const auto v = ld8(y + (long)pl[k] * C + c);
        const float wk = wt[k];
#pragma unroll
        for (int j = 0; j < 8; ++j) a[j] = fmaf(wk, get8(v, j), a[j]);
      }
      f32x8 r = ld8(xr + c);
#pragma unroll
      for (int j = 0; j < 8; ++j) r[j] = fmaf(mult, a[j], r[j]);
      st8(xr + c, r);
    }
  } else {
    for (int c = threadIdx.x; c < C; c += 256) {
      float a = 0.f;
      for (int k = 0; k < top; ++k)
        a = fmaf(wt[k], El<T>::ld(y[(long)pl[k] * C + c]), a);
      xr[c] = fmaf(mult, a, xr[c]);
    }
  }
}

// act[(m, k)] = relu(W_up[e] h[m])^2 for the k-th expert e of row m. grid
// (ceil(ff / 8), M * top); a wave takes two rows of W_up. GAIN: h is x (float32)
// under a norm with one gain. Block (0, m * top) writes ids and weights.
template <bool GAIN>
__global__ void __launch_bounds__(256)
k_moe_up_gemv(u16* __restrict__ act, int* __restrict__ ids,
              float* __restrict__ w, const float* __restrict__ logits,
              const u16* __restrict__ up, const void* __restrict__ xv,
              const float* __restrict__ gain, float eps, int E, int top,
              int ff, int C, float scale) {
  __shared__ float z[MAX_E];
  __shared__ int sid[MAX_E];
  __shared__ float sw[MAX_E];
  __shared__ float red[4];
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int m = blockIdx.y / top, k = blockIdx.y - m * top;
  for (int e = tid; e < E; e += 256) z[e] = logits[(long)m * E + e];
  for (int i = tid; i < top; i += 256) {
    sid[i] = i;
    sw[i] = 0.f;
  }
  __syncthreads();
  float sum = choose(z, E, top, tid, 256, sid, sw);
  if (blockIdx.x == 0 && k == 0) {
    sum = block_reduce_sum(sum, red) + 1e-20f;
    for (int i = tid; i < top; i += 256) {
      ids[m * top + i] = sid[i];
      w[m * top + i] = sw[i] / sum * scale;
    }
  } else {
    __syncthreads();
  }
  const int n0 = (blockIdx.x * 4 + wid) * 2;
  if (n0 >= ff) return;
  const int n1 = min(n0 + 1, ff - 1);
  const u16* we = up + (long)sid[k] * ff * C;
  const s16x8* w0 = (const s16x8*)(we + (long)n0 * C);
  const s16x8* w1 = (const s16x8*)(we + (long)n1 * C);
  float a0 = 0.f, a1 = 0.f, ss = 0.f;
  for (int i = lane; i < (C >> 3); i += 64) {
    const s16x8 v0 = w0[i], v1 = w1[i];
    if (GAIN) {
      const f32x8 x = ld8((const float*)xv + (long)m * C + i * 8);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        a0 = fmaf(x[j], bf2f((u16)v0[j]), a0);
        a1 = fmaf(x[j], bf2f((u16)v1[j]), a1);
        ss = fmaf(x[j], x[j], ss);
      }
    } else {
      const s16x8 x = ld8((const u16*)xv + (long)m * C + i * 8);
      a0 += dot8_bf16(x, v0);
      a1 += dot8_bf16(x, v1);
    }
  }
  a0 = wave_reduce_sum(a0);
  a1 = wave_reduce_sum(a1);
  if (GAIN) {
    const float inv =
        *gain / sqrtf(wave_reduce_sum(ss) / (float)C + eps);
    a0 *= inv;
    a1 *= inv;
  }
  if (lane == 0) {
    u16* dst = act + (long)blockIdx.y * ff;
    dst[n0] = El<u16>::st(relu2(a0));
    if (n1 > n0) dst[n1] = El<u16>::st(relu2(a1));
  }
}

// x[m] += mult * (W_o a[m] + sum_k w[m, k] W_down[e(m, k)] act[m, k]); Ko = 0
// leaves W_o out. The block's waves share two columns.
template <int M>
__global__ void __launch_bounds__(256)
k_moe_out_gemv(float* __restrict__ x, const u16* __restrict__ a, long as,
               const u16* __restrict__ wo, const u16* __restrict__ act,
               const int* __restrict__ ids, const float* __restrict__ w,
               const u16* __restrict__ down, int C, int Ko, int ff, int top,
               float mult) {
  __shared__ float red[4][2][M];
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int n0 = blockIdx.x * 2, n1 = min(n0 + 1, C - 1);
  float a0[M], a1[M];
#pragma unroll
  for (int m = 0; m < M; ++m) a0[m] = a1[m] = 0.f;
  const s16x8* o0 = (const s16x8*)(wo + (long)n0 * Ko);
  const s16x8* o1 = (const s16x8*)(wo + (long)n1 * Ko);
  for (int i = tid; i < (Ko >> 3); i += 256) {
    const s16x8 v0 = o0[i], v1 = o1[i];
#pragma unroll
    for (int m = 0; m < M; ++m) {
      const s16x8 xv = ld8(a + m * as + i * 8);
      a0[m] += dot8_bf16(xv, v0);
      a1[m] += dot8_bf16(xv, v1);
    }
  }
  const int nv = ff >> 3;
#pragma unroll
  for (int m = 0; m < M; ++m)
    for (int i = tid; i < top * nv; i += 256) {
      const int k = i / nv, c = i - k * nv;
      const u16* we = down + (long)ids[m * top + k] * C * ff;
      const float wk = w[m * top + k];
      const s16x8 xv = ld8(act + (long)(m * top + k) * ff + c * 8);
      a0[m] = fmaf(wk, dot8_bf16(xv, ld8(we + (long)n0 * ff + c * 8)), a0[m]);
      a1[m] = fmaf(wk, dot8_bf16(xv, ld8(we + (long)n1 * ff + c * 8)), a1[m]);
    }
#pragma unroll
  for (int m = 0; m < M; ++m) {
    a0[m] = wave_reduce_sum(a0[m]);
    a1[m] = wave_reduce_sum(a1[m]);
    if (lane == 0) {
      red[wid][0][m] = a0[m];
      red[wid][1][m] = a1[m];
    }
  }
  __syncthreads();
  if (tid >= 2 * M) return;
  const int m = tid >> 1, n = tid & 1;
  if (n == 1 && n1 == n0) return;
  x[(long)m * C + n0 + n] += mult * ((red[0][n][m] + red[1][n][m]) +
                                     (red[2][n][m] + red[3][n][m]));
}

}  // namespace

extern "C" {

void fei_moe_route(int* ids, float* w, const float* logits, int T, int E,
                   int top, float scale, hipStream_t stream) {
  hipLaunchKernelGGL(k_moe_route, dim3((T + 3) / 4), dim3(256), 0, stream, ids,
                     w, logits, T, E, top, scale);
}

void fei_moe_plan(int* order, int* place, int* tiles, int* count,
                  const int* ids, int n, int E, int top, int rows,
                  int max_tiles, hipStream_t stream) {
  hipLaunchKernelGGL(k_moe_plan, dim3(1), dim3(1024), 0, stream, order, place,
                     tiles, count, ids, n, E, top, rows, max_tiles);
}

// bits: 1 = float32, 2 = tiles of 128 slots (else 32)
void fei_moe_gemm(void* out, const void* x, const void* w, const int* order,
                  const int* tiles, const int* count, int max_tiles, int N,
                  int K, int act, int bits, hipStream_t stream) {
  if (bits & 2) {
    // 192 columns a block unless they are wasted or leave CUs without a block
    const int c6 = (N + 191) / 192, c4 = (N + 127) / 128;
    if (c6 * max_tiles >= 512 && c6 * 192 * 10 <= c4 * 128 * 11)
      launch_big<6, 2>((u16*)out, (const u16*)x, (const u16*)w, order, tiles,
                       count, max_tiles, N, K, act, stream);
    else
      launch_big<4, 2>((u16*)out, (const u16*)x, (const u16*)w, order, tiles,
                       count, max_tiles, N, K, act, stream);
    return;
  }
  const dim3 grid((N + 63) / 64, max_tiles);
#define GEMM(T, VEC)                                                        \
  hipLaunchKernelGGL((k_moe_gemm<T, VEC>), grid, dim3(256), 0, stream,      \
                     (T*)out, (const T*)x, (const T*)w, order, tiles, count, \
                     N, K, act)
  if (bits & 1) {
    if (K % 8 == 0) GEMM(float, true); else GEMM(float, false);
  } else {
    if (K % 8 == 0) GEMM(u16, true); else GEMM(u16, false);
  }
#undef GEMM
}

void fei_moe_add(float* x, const void* y, const int* place, const float* w,
                 int T, int C, int top, float mult, int f32,
                 hipStream_t stream) {
  const int vec = C % 8 == 0;
  if (f32)
    hipLaunchKernelGGL(k_moe_add<float>, dim3(T), dim3(256), 0, stream, x,
                       (const float*)y, place, w, C, top, mult, vec);
  else
    hipLaunchKernelGGL(k_moe_add<u16>, dim3(T), dim3(256), 0, stream, x,
                       (const u16*)y, place, w, C, top, mult, vec);
}

// gain_x: x is float32 under a norm with one gain, else normed bfloat16 rows.
// C % 8 == 0.
void fei_moe_up_gemv(void* act, int* ids, float* w, const float* logits,
                     const void* up, const void* x, int gain_x,
                     const float* gain, float eps, int M, int E, int top,
                     int ff, int C, float scale, hipStream_t stream) {
  const dim3 grid((ff + 7) / 8, M * top);
  if (gain_x)
    hipLaunchKernelGGL(k_moe_up_gemv<true>, grid, dim3(256), 0, stream,
                       (u16*)act, ids, w, logits, (const u16*)up, x, gain,
                       eps, E, top, ff, C, scale);
  else
    hipLaunchKernelGGL(k_moe_up_gemv<false>, grid, dim3(256), 0, stream,
                       (u16*)act, ids, w, logits, (const u16*)up, x, gain,
                       eps, E, top, ff, C, scale);
}

// M in {1, 2, 4, 8}; Ko, ff % 8 == 0.
void fei_moe_out_gemv(float* x, const void* a, long as, const void* wo,
                      const void* act, const int* ids, const float* w,
                      const void* down, int M, int C, int Ko, int ff, int top,
                      float mult, hipStream_t stream) {
  const dim3 grid((C + 1) / 2);
#define OUT(MV)                                                             \
  hipLaunchKernelGGL(k_moe_out_gemv<MV>, grid, dim3(256), 0, stream, x,     \
                     (const u16*)a, as, (const u16*)wo, (const u16*)act,    \
                     ids, w, (const u16*)down, C, Ko, ff, top, mult)
  switch (M) {
    case 1: OUT(1); break;
    case 2: OUT(2); break;
    case 4: OUT(4); break;
    case 8: OUT(8); break;
    default: break;
  }
#undef OUT
}

}  // extern "C"
