// Shared parts of the recurrences with matrix states (linscan.hip, delta.hip).
#pragma once
#include "common.h"

namespace lmx {

__device__ __forceinline__ float softplus_f(float x) { return x > 20.f ? x : log1pf(expf(x)); }

constexpr float SCAN_LOG2E = 1.4426950408889634f;

// columns per workgroup: the largest power of two up to `want_pt` whose rows
// per thread fit the register tile (16 x 4 or 8 x 1 values)
static inline bool recurrent_shape(int N, int P, int want_pt, int* vec, int* pt, int* rpt) {
  *vec = P % 4 == 0 ? 4 : 1;
  int t = 16;
  while (t < P && t < want_pt) t *= 2;
  for (;; t /= 2) {
    const int ncol = t / *vec;
    if (ncol < 1 || t < 4) return false;
    const int kr = 256 / ncol, r = (N + kr - 1) / kr;
    if (r <= (*vec == 4 ? 16 : 8)) { *pt = t; *rpt = r; return true; }
  }
}

typedef uint32_t u32x4_t __attribute__((ext_vector_type(4)));
typedef uint32_t u32x2_t __attribute__((ext_vector_type(2)));

// (a, b) as packed bf16 pairs: hi + lo = the values to within 2^-17
__device__ __forceinline__ void split2(float a, float b, uint32_t& hi, uint32_t& lo) {
  hi = pack_bf16x2(a, b);
  lo = pack_bf16x2(a - __uint_as_float(hi << 16), b - __uint_as_float(hi & 0xffff0000u));
}

// Transposed LDS image [rows][64 tokens]: 16-B pieces (8 tokens) of a row are
// XOR-permuted by the row so that both the 8-B transposing stores (16 row
// groups x 4 token quads per wave) and the 16-B fragment reads (16 rows x 4
// pieces) spread evenly over the banks.
__device__ __forceinline__ int tr_swz(int row) {
  return ((row & 3) | ((row >> 1) & 4)) ^ ((row >> 4) & 7);
}

}  // namespace lmx
