// What a skinny matrix product does with its float32 sums.
#pragma once
#include "fei_common.h"

enum { EPI_BF16 = 0, EPI_F32 = 1, EPI_RES = 2 };

struct Epilogue {
  const float* bias;   // per column, may be null
  float scale;
  float cap;           // 0: no softcap
};

__device__ __forceinline__ float softcap(float v, float scale, float cap) {
  v *= scale;
  return cap > 0.f ? cap * tanhf(v / cap) : v;
}

template <int EPI>
__device__ __forceinline__ void epilogue(void* out, long at, int col, float v,
                                         const Epilogue& ep) {
  if (EPI == EPI_BF16) {
    ((u16*)out)[at] = f2bf(v);
  } else if (EPI == EPI_RES) {
    ((float*)out)[at] += v;
  } else {
    v = softcap(v, ep.scale, ep.cap);
    ((float*)out)[at] = ep.bias ? v + ep.bias[col] : v;
  }
}
