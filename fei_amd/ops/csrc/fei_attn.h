// What the attention kernels over a paged cache of rows share.
#pragma once
#include "fei_mma.h"

// First key that position ``pos`` sees; window 0 = all.
__device__ __forceinline__ int first_key(int pos, int window) {
  return window > 0 && pos >= window ? pos - window + 1 : 0;
}

// Cached row of a position of a sequence; blocks of 2^bs_log rows.
__device__ __forceinline__ long cache_row(const int* __restrict__ table,
                                          int W, int seq, int pos,
                                          int bs_log) {
  return ((long)table[(long)seq * W + (pos >> bs_log)] << bs_log) +
         (pos & ((1 << bs_log) - 1));
}

// A float32 weight as operand: one part for float, a high and a low one
// (about 16 bits together) for bfloat16.
template <typename T> struct Parts { static constexpr int n = 1; };
template <> struct Parts<u16> { static constexpr int n = 2; };

template <typename T>
__device__ __forceinline__ T part_of(float v, int i) {
  const T hi = El<T>::st(v);
  return i == 0 ? hi : El<T>::st(v - El<T>::ld(hi));
}

// Eight weights as fragments, two conversions at a time.
__device__ __forceinline__ void weight_parts(const float (&v)[8],
                                             s16x8 (&p)[2]) {
  typedef __attribute__((ext_vector_type(2))) __bf16 bf16x2;
  typedef __attribute__((ext_vector_type(4))) u32 u32x4;
  u32x4 hi, lo;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const f32x2 x = {v[2 * i], v[2 * i + 1]};
    hi[i] = __builtin_bit_cast(u32, __builtin_convertvector(x, bf16x2));
    const f32x2 y = {x[0] - __builtin_bit_cast(float, hi[i] << 16),
                     x[1] - __builtin_bit_cast(float, hi[i] & 0xffff0000u)};
    lo[i] = __builtin_bit_cast(u32, __builtin_convertvector(y, bf16x2));
  }
  p[0] = __builtin_bit_cast(s16x8, hi);
  p[1] = __builtin_bit_cast(s16x8, lo);
}
__device__ __forceinline__ void weight_parts(const float (&v)[8],
                                             f32x8 (&p)[1]) {
#pragma unroll
  for (int i = 0; i < 8; ++i) p[0][i] = v[i];
}

// Place of (column, key) in a transposed value tile: 64 keys a column in
// blocks of 8, the block index permuted by the column so that neither the
// stores (lanes along columns) nor the reads (16 columns, one block) pile up
// on a bank.
__device__ __forceinline__ int vt_at(int col, int key) {
  return col * 64 + ((((key >> 3) ^ col ^ (col >> 3)) & 7) << 3) + (key & 7);
}
