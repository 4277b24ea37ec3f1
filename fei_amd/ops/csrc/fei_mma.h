// Matrix-core tiles that read the same for bfloat16 and float32 operands.
//
// A fragment is the lane's 8 elements k = 8*(lane/16) .. +7 of row (A) or
// column (B) lane%16 of a 16x32 tile. bfloat16: one mfma_f32_16x16x32_bf16.
// float32: eight mfma_f32_16x16x4_f32, the j-th over element j of all four
// lane groups (any order of k is right as long as A and B share it), so the
// products and sums are float32 throughout.
// The result is C[4*(lane/16) + r][lane%16], r = 0..3.
#pragma once
#include "fei_common.h"

typedef __attribute__((ext_vector_type(8))) float f32x8;

__device__ __forceinline__ f32x4 mma(s16x8 a, s16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ f32x4 mma(f32x8 a, f32x8 b, f32x4 c) {
#pragma unroll
  for (int j = 0; j < 8; ++j)
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[j], b[j], c, 0, 0, 0);
  return c;
}

// Element type of rows in memory and LDS.
template <typename T> struct El;
template <> struct El<u16> {
  typedef s16x8 frag;
  static __device__ __forceinline__ float ld(u16 v) { return bf2f(v); }
  // the hardware's conversion, round to nearest even
  static __device__ __forceinline__ u16 st(float v) {
    return __builtin_bit_cast(u16, (__bf16)v);
  }
  static __device__ __forceinline__ float ex(float x) { return __expf(x); }
  // exp(x) of an x that was scaled by ``base``
  static constexpr float base = 1.44269504088896340736f;   // log2(e)
  static __device__ __forceinline__ float exb(float x) {
    return __builtin_amdgcn_exp2f(x);
  }
  static __device__ __forceinline__ float ln(float x) { return __logf(x); }
  static __device__ __forceinline__ float inv(float x) {
    return __builtin_amdgcn_rcpf(x);
  }
};
template <> struct El<float> {
  typedef f32x8 frag;
  static __device__ __forceinline__ float ld(float v) { return v; }
  static __device__ __forceinline__ float st(float v) { return v; }
  static __device__ __forceinline__ float ex(float x) { return expf(x); }
  static constexpr float base = 1.f;
  static __device__ __forceinline__ float exb(float x) { return expf(x); }
  static __device__ __forceinline__ float ln(float x) { return logf(x); }
  static __device__ __forceinline__ float inv(float x) { return 1.f / x; }
};

// 8 consecutive elements at p (16-byte aligned in LDS and, where used, in
// memory).
__device__ __forceinline__ s16x8 ld8(const u16* p) { return *(const s16x8*)p; }
__device__ __forceinline__ f32x8 ld8(const float* p) {
  const f32x4 a = *(const f32x4*)p, b = *(const f32x4*)(p + 4);
  return f32x8{a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
}
__device__ __forceinline__ void st8(u16* p, s16x8 v) { *(s16x8*)p = v; }
__device__ __forceinline__ void st8(float* p, f32x8 v) {
  *(f32x4*)p = f32x4{v[0], v[1], v[2], v[3]};
  *(f32x4*)(p + 4) = f32x4{v[4], v[5], v[6], v[7]};
}
__device__ __forceinline__ float get8(s16x8 v, int j) { return bf2f((u16)v[j]); }
__device__ __forceinline__ float get8(f32x8 v, int j) { return v[j]; }

// Reductions over the 16 lanes of a DPP row (lanes 16i .. 16i+15), by
// rotations: every lane gets the result, no LDS traffic.
template <int N>
__device__ __forceinline__ float row_ror(float v) {
  return __builtin_bit_cast(
      float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v),
                                         0x120 + N, 0xf, 0xf, true));
}
__device__ __forceinline__ float row16_max(float v) {
  v = fmaxf(v, row_ror<8>(v));
  v = fmaxf(v, row_ror<4>(v));
  v = fmaxf(v, row_ror<2>(v));
  return fmaxf(v, row_ror<1>(v));
}
__device__ __forceinline__ float row16_sum(float v) {
  v += row_ror<8>(v);
  v += row_ror<4>(v);
  v += row_ror<2>(v);
  return v + row_ror<1>(v);
}

// Precise sigmoid and silu.
__device__ __forceinline__ float sigmoid_f(float x) {
  return 1.f / (1.f + expf(-x));
}
