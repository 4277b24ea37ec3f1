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

// Place of (column, key) in a transposed value tile: 64 keys a column in
// blocks of 8, the block index permuted by the column so that neither the
// stores (lanes along columns) nor the reads (16 columns, one block) pile up
// on a bank.
__device__ __forceinline__ int vt_at(int col, int key) {
  return col * 64 + ((((key >> 3) ^ col ^ (col >> 3)) & 7) << 3) + (key & 7);
}
