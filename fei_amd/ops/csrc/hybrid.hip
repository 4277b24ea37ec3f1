// Row-wise kernels and skinny products of decoders made of unlike layers
// (models/tobarax.py, models/bokenex.py): a float32 residual, two norms of the same rows, one
// stacked product for everything a layer reads, one product over the
// concatenated mixer and feed-forward outputs that adds to the residual.
// T is the element type of rows: u16 (bfloat16 bits) or float.
#include "fei_common.h"
#include "fei_epilogue.h"
#include "fei_mma.h"

namespace {

// o1 = rms(x) * w1, o2 = rms(x) * w2 (o2 may be null). One block per row.
template <typename T>
__global__ void __launch_bounds__(256)
k_norm_pair(T* __restrict__ o1, T* __restrict__ o2,
            const float* __restrict__ x, const float* __restrict__ w1,
            const float* __restrict__ w2, int rows, int C, float eps) {
  __shared__ float red[4];
  const bool vec = (C & 3) == 0;
  for (int row = blockIdx.x; row < rows; row += gridDim.x) {
    const float* xr = x + (long)row * C;
    float ss = 0.f;
    if (vec) {
      for (int i = threadIdx.x; i < (C >> 2); i += blockDim.x) {
        const f32x4 v = ((const f32x4*)xr)[i];
#pragma unroll
        for (int j = 0; j < 4; ++j) ss = fmaf(v[j], v[j], ss);
      }
    } else {
      for (int i = threadIdx.x; i < C; i += blockDim.x)
        ss = fmaf(xr[i], xr[i], ss);
    }
    ss = block_reduce_sum(ss, red);
    const float inv = 1.f / sqrtf(ss / (float)C + eps);
    T* r1 = o1 + (long)row * C;
    T* r2 = o2 ? o2 + (long)row * C : nullptr;
    if (vec) {
      for (int i = threadIdx.x; i < (C >> 2); i += blockDim.x) {
        const f32x4 v = ((const f32x4*)xr)[i];
        const f32x4 a = ((const f32x4*)w1)[i];
        T t[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) t[j] = El<T>::st(v[j] * inv * a[j]);
        __builtin_memcpy(r1 + i * 4, t, sizeof(t));
        if (r2) {
          const f32x4 b = ((const f32x4*)w2)[i];
#pragma unroll
          for (int j = 0; j < 4; ++j) t[j] = El<T>::st(v[j] * inv * b[j]);
          __builtin_memcpy(r2 + i * 4, t, sizeof(t));
        }
      }
    } else {
      for (int i = threadIdx.x; i < C; i += blockDim.x) {
        const float y = xr[i] * inv;
        r1[i] = El<T>::st(y * w1[i]);
        if (r2) r2[i] = El<T>::st(y * w2[i]);
      }
    }
    __syncthreads();
  }
}

template <typename T>
__global__ void __launch_bounds__(256)
k_cat_cast(T* __restrict__ out, const float* __restrict__ x,
           const float* __restrict__ y, long n, int C) {
  for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < n;
       i += (long)gridDim.x * blockDim.x) {
    const long row = i / (2 * C);
    const int c = (int)(i - row * 2 * C);
    out[i] = El<T>::st(c < C ? x[row * C + c] : y[row * C + c - C]);
  }
}

// act[row, i] = silu(gu[row, i]) * gu[row, ff + i]
template <typename T>
__global__ void __launch_bounds__(256)
k_swiglu_rows(T* __restrict__ act, long as, const T* __restrict__ gu, long gs,
              int rows, int ff, int vec) {
  if (vec) {
    const int nv = ff >> 3;
    for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
         i < (long)rows * nv; i += (long)gridDim.x * blockDim.x) {
      const long row = i / nv;
      const int c = (int)(i - row * nv) * 8;
      const auto g = ld8(gu + row * gs + c);
      const auto u = ld8(gu + row * gs + ff + c);
      typename El<T>::frag o;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float gf = get8(g, j);
        o[j] = El<T>::st(gf / (1.f + El<T>::ex(-gf)) * get8(u, j));
      }
      st8(act + row * as + c, o);
    }
  } else {
    for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
         i < (long)rows * ff; i += (long)gridDim.x * blockDim.x) {
      const long row = i / ff;
      const int c = (int)(i - row * ff);
      const float g = El<T>::ld(gu[row * gs + c]);
      act[row * as + c] = El<T>::st(g / (1.f + El<T>::ex(-g)) *
                                    El<T>::ld(gu[row * gs + ff + c]));
    }
  }
}

__global__ void __launch_bounds__(256)
k_softcap(float* __restrict__ y, long n, float scale, float cap) {
  for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < n;
       i += (long)gridDim.x * blockDim.x)
    y[i] = softcap(y[i], scale, cap);
}

// Two weight rows, streamed 16 bytes a lane by the lanes of ``step`` / 64
// waves; the sums are this wave's. x comes from L1/L2.
template <int M, bool NT>
__device__ __forceinline__ void two_rows(const u16* __restrict__ x,
                                         const u16* __restrict__ w0,
                                         const u16* __restrict__ w1, int K,
                                         int first, int step, float* a0,
                                         float* a1) {
#pragma unroll
  for (int m = 0; m < M; ++m) a0[m] = a1[m] = 0.f;
  const int nv = K >> 3;
  for (int i = first; i < nv; i += step) {
    const s16x8 v0 = NT ? __builtin_nontemporal_load((const s16x8*)w0 + i)
                        : ((const s16x8*)w0)[i];
    const s16x8 v1 = NT ? __builtin_nontemporal_load((const s16x8*)w1 + i)
                        : ((const s16x8*)w1)[i];
#pragma unroll
    for (int m = 0; m < M; ++m) {
      const s16x8 xv = ((const s16x8*)(x + (long)m * K))[i];
      a0[m] += dot8_bf16(xv, v0);
      a1[m] += dot8_bf16(xv, v1);
    }
  }
#pragma unroll
  for (int m = 0; m < M; ++m) {
    a0[m] = wave_reduce_sum(a0[m]);
    a1[m] = wave_reduce_sum(a1[m]);
  }
}

// Everything a layer reads from its two normed inputs, in one launch:
// proj[m, n] = x1[m] . w[n] for n < n_mix, and for each i < ff
// act[m, i] = silu(x2[m] . w[n_mix + i]) * (x2[m] . w[n_mix + ff + i]).
// A wave takes two mixer rows or one gate/up pair.
template <int M, bool NT>
__global__ void __launch_bounds__(256)
k_gemv_mix_in(u16* __restrict__ proj, u16* __restrict__ act,
              const u16* __restrict__ x1, const u16* __restrict__ x2,
              const u16* __restrict__ w, long as, int n_mix, int ff, int K) {
  const int lane = threadIdx.x & 63;
  const int u = blockIdx.x * 4 + (threadIdx.x >> 6);
  const int units = (n_mix + 1) / 2;
  float a0[M], a1[M];
  if (u < units) {
    const int r0 = 2 * u, r1 = min(2 * u + 1, n_mix - 1);
    two_rows<M, NT>(x1, w + (long)r0 * K, w + (long)r1 * K, K, lane, 64, a0,
                    a1);
    if (lane == 0) {
#pragma unroll
      for (int m = 0; m < M; ++m) {
        proj[(long)m * n_mix + r0] = f2bf(a0[m]);
        if (r1 > r0) proj[(long)m * n_mix + r1] = f2bf(a1[m]);
      }
    }
  } else if (u - units < ff) {
    const int i = u - units;
    two_rows<M, NT>(x2, w + (long)(n_mix + i) * K,
                    w + (long)(n_mix + ff + i) * K, K, lane, 64, a0, a1);
    if (lane == 0) {
#pragma unroll
      for (int m = 0; m < M; ++m) {
        const float g = a0[m];
        act[(long)m * as + i] = f2bf(g / (1.f + __expf(-g)) * a1[m]);
      }
    }
  }
}

// out rows by an epilogue, two weight rows at a time. KSPLIT 1: a wave takes
// two whole rows. KSPLIT 4: the block's waves share two rows, for products
// with too few rows to fill the chip.
template <int M, bool NT, int EPI, int KSPLIT>
__global__ void __launch_bounds__(256)
k_gemv_f32(float* __restrict__ out, const u16* __restrict__ x,
           const u16* __restrict__ w, int N, int K, Epilogue ep) {
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int n0 = (KSPLIT == 1 ? blockIdx.x * 4 + wid : blockIdx.x) * 2;
  if (n0 >= N) return;
  const int n1 = min(n0 + 1, N - 1);
  float a0[M], a1[M];
  two_rows<M, NT>(x, w + (long)n0 * K, w + (long)n1 * K, K,
                  KSPLIT == 1 ? lane : wid * 64 + lane, KSPLIT * 64, a0, a1);
  if (KSPLIT > 1) {
    __shared__ float red[4][2][M];
    if (lane == 0) {
#pragma unroll
      for (int m = 0; m < M; ++m) {
        red[wid][0][m] = a0[m];
        red[wid][1][m] = a1[m];
      }
    }
    __syncthreads();
    if (threadIdx.x >= 2 * M) return;
    const int m = threadIdx.x >> 1, n = threadIdx.x & 1;
    if (n == 1 && n1 == n0) return;
    epilogue<EPI>(out, m, N, n0 + n,
                  (red[0][n][m] + red[1][n][m]) + (red[2][n][m] + red[3][n][m]),
                  ep);
  } else if (lane == 0) {
#pragma unroll
    for (int m = 0; m < M; ++m) {
      epilogue<EPI>(out, m, N, n0, a0[m], ep);
      if (n1 > n0) epilogue<EPI>(out, m, N, n1, a1[m], ep);
    }
  }
}

// The same of rows under an RMS norm with one gain: x float32 as it is, the
// sums times gain / rms(x).
template <int M, int EPI, int KSPLIT>
__global__ void __launch_bounds__(256)
k_gemv_gain(void* __restrict__ out, const float* __restrict__ x,
            const u16* __restrict__ w, const float* __restrict__ gain,
            float eps, int N, int K, Epilogue ep) {
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int n0 = (KSPLIT == 1 ? blockIdx.x * 4 + wid : blockIdx.x) * 2;
  if (n0 >= N) return;
  const int n1 = min(n0 + 1, N - 1);
  const s16x8* w0 = (const s16x8*)(w + (long)n0 * K);
  const s16x8* w1 = (const s16x8*)(w + (long)n1 * K);
  float a[3][M];                           // two rows, sum of squares
#pragma unroll
  for (int m = 0; m < M; ++m) a[0][m] = a[1][m] = a[2][m] = 0.f;
  for (int i = KSPLIT == 1 ? lane : threadIdx.x; i < (K >> 3);
       i += KSPLIT * 64) {
    const s16x8 v0 = __builtin_nontemporal_load(w0 + i);
    const s16x8 v1 = __builtin_nontemporal_load(w1 + i);
#pragma unroll
    for (int m = 0; m < M; ++m) {
      const f32x8 xv = ld8(x + (long)m * K + i * 8);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        a[0][m] = fmaf(xv[j], bf2f((u16)v0[j]), a[0][m]);
        a[1][m] = fmaf(xv[j], bf2f((u16)v1[j]), a[1][m]);
        a[2][m] = fmaf(xv[j], xv[j], a[2][m]);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < 3; ++i)
#pragma unroll
    for (int m = 0; m < M; ++m) a[i][m] = wave_reduce_sum(a[i][m]);
  if (KSPLIT > 1) {
    __shared__ float red[4][3][M];
    if (lane == 0) {
#pragma unroll
      for (int i = 0; i < 3; ++i)
#pragma unroll
        for (int m = 0; m < M; ++m) red[wid][i][m] = a[i][m];
    }
    __syncthreads();
    if (threadIdx.x >= 2 * M) return;
    const int m = threadIdx.x >> 1, n = threadIdx.x & 1;
    if (n == 1 && n1 == n0) return;
    const float ss = (red[0][2][m] + red[1][2][m]) +
                     (red[2][2][m] + red[3][2][m]);
    epilogue<EPI>(out, m, N, n0 + n,
                  ((red[0][n][m] + red[1][n][m]) +
                   (red[2][n][m] + red[3][n][m])) *
                      (*gain / sqrtf(ss / (float)K + eps)), ep);
  } else if (lane == 0) {
#pragma unroll
    for (int m = 0; m < M; ++m) {
      const float inv = *gain / sqrtf(a[2][m] / (float)K + eps);
      epilogue<EPI>(out, m, N, n0, a[0][m] * inv, ep);
      if (n1 > n0) epilogue<EPI>(out, m, N, n1, a[1][m] * inv, ep);
    }
  }
}

// out[t] = emb[tok[t]] + pos_emb[pos[t]]
template <typename T, typename I>
__global__ void __launch_bounds__(256)
k_embed_pos(float* __restrict__ out, const I* __restrict__ tok,
            const int* __restrict__ pos, const T* __restrict__ emb,
            const T* __restrict__ pos_emb, int C) {
  const int t = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
  if (c < C)
    out[(long)t * C + c] = El<T>::ld(emb[(long)tok[t] * C + c]) +
                           El<T>::ld(pos_emb[(long)pos[t] * C + c]);
}

// act = relu(up)^2
template <typename T>
__global__ void __launch_bounds__(256)
k_relu2_rows(T* __restrict__ act, long as, const T* __restrict__ up, long us,
             int rows, int ff, int vec) {
  const int nv = vec ? ff >> 3 : ff;
  for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
       i < (long)rows * nv; i += (long)gridDim.x * blockDim.x) {
    const long row = i / nv;
    const int c = (int)(i - row * nv);
    if (vec) {
      const auto u = ld8(up + row * us + c * 8);
      typename El<T>::frag o;
#pragma unroll
      for (int j = 0; j < 8; ++j) o[j] = El<T>::st(relu2(get8(u, j)));
      st8(act + row * as + c * 8, o);
    } else {
      act[row * as + c] = El<T>::st(relu2(El<T>::ld(up[row * us + c])));
    }
  }
}

inline int grid_for(long n, int per) {
  const long g = (n + per - 1) / per;
  return (int)(g < 1 ? 1 : (g > 4096 ? 4096 : g));
}

}  // namespace

extern "C" {

void fei_norm_pair(void* o1, void* o2, const float* x, const float* w1,
                   const float* w2, int rows, int C, float eps, int f32,
                   hipStream_t stream) {
  const dim3 grid(rows < 4096 ? rows : 4096);
  if (f32)
    hipLaunchKernelGGL(k_norm_pair<float>, grid, dim3(256), 0, stream,
                       (float*)o1, (float*)o2, x, w1, w2, rows, C, eps);
  else
    hipLaunchKernelGGL(k_norm_pair<u16>, grid, dim3(256), 0, stream,
                       (u16*)o1, (u16*)o2, x, w1, w2, rows, C, eps);
}

void fei_cat_cast(void* out, const float* x, const float* y, int rows, int C,
                  int f32, hipStream_t stream) {
  const long n = (long)rows * 2 * C;
  if (f32)
    hipLaunchKernelGGL(k_cat_cast<float>, dim3(grid_for(n, 256)), dim3(256),
                       0, stream, (float*)out, x, y, n, C);
  else
    hipLaunchKernelGGL(k_cat_cast<u16>, dim3(grid_for(n, 256)), dim3(256), 0,
                       stream, (u16*)out, x, y, n, C);
}

void fei_swiglu_rows(void* act, long as, const void* gu, long gs, int rows,
                     int ff, int f32, hipStream_t stream) {
  const int vec = ff % 8 == 0 && as % 8 == 0 && gs % 8 == 0 &&
                  (size_t)act % 16 == 0 && (size_t)gu % 16 == 0;
  const dim3 grid(grid_for((long)rows * ff, vec ? 2048 : 256));
  if (f32)
    hipLaunchKernelGGL(k_swiglu_rows<float>, grid, dim3(256), 0, stream,
                       (float*)act, as, (const float*)gu, gs, rows, ff, vec);
  else
    hipLaunchKernelGGL(k_swiglu_rows<u16>, grid, dim3(256), 0, stream,
                       (u16*)act, as, (const u16*)gu, gs, rows, ff, vec);
}

// bits: 1 = float32 rows, 2 = 64-bit token ids
void fei_embed_pos(float* out, const void* tok, const int* pos,
                   const void* emb, const void* pos_emb, int T, int C,
                   int bits, hipStream_t stream) {
  const dim3 grid(T, (C + 255) / 256);
#define EMB(E, I)                                                           \
  hipLaunchKernelGGL((k_embed_pos<E, I>), grid, dim3(256), 0, stream, out,  \
                     (const I*)tok, pos, (const E*)emb, (const E*)pos_emb, C)
  switch (bits) {
    case 0: EMB(u16, int); break;
    case 1: EMB(float, int); break;
    case 2: EMB(u16, long); break;
    default: EMB(float, long); break;
  }
#undef EMB
}

void fei_relu2_rows(void* act, long as, const void* up, long us, int rows,
                    int ff, int f32, hipStream_t stream) {
  const int vec = ff % 8 == 0 && as % 8 == 0 && us % 8 == 0 &&
                  (size_t)act % 16 == 0 && (size_t)up % 16 == 0;
  const dim3 grid(grid_for((long)rows * ff, vec ? 2048 : 256));
  if (f32)
    hipLaunchKernelGGL(k_relu2_rows<float>, grid, dim3(256), 0, stream,
                       (float*)act, as, (const float*)up, us, rows, ff, vec);
  else
    hipLaunchKernelGGL(k_relu2_rows<u16>, grid, dim3(256), 0, stream,
                       (u16*)act, as, (const u16*)up, us, rows, ff, vec);
}

void fei_softcap(float* y, long n, float scale, float cap,
                 hipStream_t stream) {
  hipLaunchKernelGGL(k_softcap, dim3(grid_for(n, 1024)), dim3(256), 0, stream,
                     y, n, scale, cap);
}

#define BY_M(M_, CALL)            \
  switch (M_) {                   \
    case 1: CALL(1); break;       \
    case 2: CALL(2); break;       \
    case 4: CALL(4); break;       \
    case 8: CALL(8); break;       \
    default: break;               \
  }

// M in {1, 2, 4, 8}, K % 8 == 0 (the caller checks).
void fei_gemv_mix_in(void* proj, void* act, const void* x1, const void* x2,
                     const void* w, long as, int M, int n_mix, int ff, int K,
                     int nt, hipStream_t stream) {
  const dim3 grid(((n_mix + 1) / 2 + ff + 3) / 4);
#define CALL(MV)                                                            \
  if (nt)                                                                   \
    hipLaunchKernelGGL((k_gemv_mix_in<MV, true>), grid, dim3(256), 0,       \
                       stream, (u16*)proj, (u16*)act, (const u16*)x1,       \
                       (const u16*)x2, (const u16*)w, as, n_mix, ff, K);    \
  else                                                                      \
    hipLaunchKernelGGL((k_gemv_mix_in<MV, false>), grid, dim3(256), 0,      \
                       stream, (u16*)proj, (u16*)act, (const u16*)x1,       \
                       (const u16*)x2, (const u16*)w, as, n_mix, ff, K)
  BY_M(M, CALL)
#undef CALL
}

// Products of one or two rows under a norm with one gain, K % 8 == 0.
#define GAIN(EPI)                                                           \
  do {                                                                      \
    if (M == 1) {                                                           \
      if (share) GAIN_(1, EPI, 4); else GAIN_(1, EPI, 1);                   \
    } else if (M == 2) {                                                    \
      if (share) GAIN_(2, EPI, 4); else GAIN_(2, EPI, 1);                   \
    }                                                                       \
  } while (0)
#define GAIN_(MV, EPI, KSP)                                                 \
  hipLaunchKernelGGL((k_gemv_gain<MV, EPI, KSP>), grid, dim3(256), 0,       \
                     stream, out, x, (const u16*)w, gain, eps, N, K, ep)

void fei_gemv_gain(void* out, const float* x, const void* w,
                   const float* gain, float eps, int M, int N, int K,
                   hipStream_t stream) {
  const bool share = N < 8192;
  const dim3 grid(share ? (N + 1) / 2 : (N + 7) / 8);
  const Epilogue ep{nullptr, 1.f, 0.f};
  GAIN(EPI_F32);
}

// All products of a parallel layer's input (see EPI_PARALLEL).
void fei_gemv_parallel_in(void* out, float* router, const float* x,
                          const void* w, const float* gain, float eps,
                          void* act, long as, int M, int n_mix, int n_router,
                          int N, int K, hipStream_t stream) {
  const bool share = N < 8192;
  const dim3 grid(share ? (N + 1) / 2 : (N + 7) / 8);
  const Epilogue ep{nullptr, 1.f,    0.f,       n_mix,
                    n_router, router, (u16*)act, as};
  GAIN(EPI_PARALLEL);
}
#undef GAIN
#undef GAIN_

// residual != 0: out += scale x w^T; else out = softcap(x w^T * scale, cap) + bias.
void fei_gemv_f32(void* out, const void* x, const void* w, const float* bias,
                  int M, int N, int K, int residual, float scale, float cap,
                  int nt, hipStream_t stream) {
  const bool share = N < 8192;             // rows alone do not fill the chip
  const dim3 grid(share ? (N + 1) / 2 : (N + 7) / 8);
  const Epilogue ep{bias, scale, cap};
#define LAUNCH(MV, NTV, EPI, KSP)                                           \
  hipLaunchKernelGGL((k_gemv_f32<MV, NTV, EPI, KSP>), grid, dim3(256), 0,   \
                     stream, (float*)out, (const u16*)x, (const u16*)w, N,  \
                     K, ep)
#define BY_NT(MV, EPI, KSP)                                                 \
  do {                                                                      \
    if (nt) LAUNCH(MV, true, EPI, KSP); else LAUNCH(MV, false, EPI, KSP);   \
  } while (0)
#define CALL(MV)                                                            \
  if (residual) {                                                           \
    if (share) BY_NT(MV, EPI_RES, 4); else BY_NT(MV, EPI_RES, 1);           \
  } else {                                                                  \
    if (share) BY_NT(MV, EPI_F32, 4); else BY_NT(MV, EPI_F32, 1);           \
  }
  BY_M(M, CALL)
#undef CALL
#undef BY_NT
#undef LAUNCH
}

}  // extern "C"
