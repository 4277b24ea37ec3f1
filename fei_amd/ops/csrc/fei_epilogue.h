// What a skinny matrix product does with its float32 sums.
#pragma once
#include "fei_common.h"

enum { EPI_BF16 = 0, EPI_F32 = 1, EPI_RES = 2, EPI_PARALLEL = 3 };

struct Epilogue {
  const float* bias;   // per column, may be null
  float scale;
  float cap;           // 0: no softcap
  // EPI_PARALLEL: n_mix columns go to out, the next n_router to router, of
  // the rest relu(.)^2 to act, whose rows are ``as`` apart
  int n_mix, n_router;
  float* router;
  u16* act;
  long as;
};

__device__ __forceinline__ float softcap(float v, float scale, float cap) {
  v *= scale;
  return cap > 0.f ? cap * tanhf(v / cap) : v;
}

__device__ __forceinline__ float relu2(float v) {
  v = fmaxf(v, 0.f);
  return v * v;
}

// N: columns of out
template <int EPI>
__device__ __forceinline__ void epilogue(void* out, int row, int N, int col,
                                         float v, const Epilogue& ep) {
  const long at = (long)row * N + col;
  if (EPI == EPI_BF16) {
    ((u16*)out)[at] = f2bf(v);
  } else if (EPI == EPI_RES) {
    ((float*)out)[at] += v * ep.scale;
  } else if (EPI == EPI_F32) {
    v = softcap(v, ep.scale, ep.cap);
    ((float*)out)[at] = ep.bias ? v + ep.bias[col] : v;
  } else if (col < ep.n_mix) {
    ((u16*)out)[(long)row * ep.n_mix + col] = f2bf(v);
  } else if (col < ep.n_mix + ep.n_router) {
    ep.router[(long)row * ep.n_router + col - ep.n_mix] = v;
  } else {
    ep.act[row * ep.as + col - ep.n_mix - ep.n_router] = f2bf(relu2(v));
  }
}
