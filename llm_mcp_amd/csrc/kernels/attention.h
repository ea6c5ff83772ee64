// Shared parts of the paged attention kernels (attention.hip, talk.hip).
#pragma once
#include "common.h"

namespace lmx {

constexpr int BS = 32;   // KV page (block) size in tokens
constexpr float LOG2E = 1.4426950408889634f;

// max / sum over the 4 lanes c, c+16, c+32, c+48 (one MFMA column's 4 row
// groups) with v_permlane16_swap / v_permlane32_swap: VALU lane exchanges
// instead of two ds_bpermute round trips through the LDS unit on the softmax's
// serial chain.  permlane16_swap(x, x) yields {rows 0,0,2,2 ; rows 1,1,3,3} of
// x (16-lane rows), so op(first, second) is the xor-16 reduction; the 32-lane
// form does the same across halves.
// v_max_f32 as one instruction (fmaxf on values hipcc cannot prove canonical
// -- MFMA results, lane swaps -- gets a canonicalising v_max per operand)
__device__ __forceinline__ float max2f(float a, float b) {
  float r;
  asm("v_max_f32 %0, %1, %2" : "=v"(r) : "v"(a), "v"(b));
  return r;
}

// v_max3_f32 as one instruction (the same canonicalisation otherwise doubles
// the row-max VALU of the softmax)
__device__ __forceinline__ float max3f(float a, float b, float c) {
  float r;
  asm("v_max3_f32 %0, %1, %2, %3" : "=v"(r) : "v"(a), "v"(b), "v"(c));
  return r;
}

__device__ __forceinline__ float col4_max(float x) {
  const unsigned u = __float_as_uint(x);
  const auto a = __builtin_amdgcn_permlane16_swap(u, u, false, false);
  x = max2f(__uint_as_float(a[0]), __uint_as_float(a[1]));
  const unsigned v = __float_as_uint(x);
  const auto b = __builtin_amdgcn_permlane32_swap(v, v, false, false);
  return max2f(__uint_as_float(b[0]), __uint_as_float(b[1]));
}

__device__ __forceinline__ float col4_sum(float x) {
  const unsigned u = __float_as_uint(x);
  const auto a = __builtin_amdgcn_permlane16_swap(u, u, false, false);
  x = __uint_as_float(a[0]) + __uint_as_float(a[1]);
  const unsigned v = __float_as_uint(x);
  const auto b = __builtin_amdgcn_permlane32_swap(v, v, false, false);
  return __uint_as_float(b[0]) + __uint_as_float(b[1]);
}

// K/V page loads; NTL: non-temporal (the decode step reads each page once per
// layer, with the whole model streamed between two reads of it)
template <bool NTL>
__device__ __forceinline__ bf16x8_t kv_frag16B(const bf16_t* p) {
  if constexpr (NTL) return __builtin_nontemporal_load(reinterpret_cast<const bf16x8_t*>(p));
  else return load_frag16B(p);
}

template <bool NTL>
__device__ __forceinline__ bf16x8_t kv_frag_2x8B(const bf16_t* p0, const bf16_t* p1) {
  if constexpr (NTL) {
    const bf16x4_t a = __builtin_nontemporal_load(reinterpret_cast<const bf16x4_t*>(p0));
    const bf16x4_t b = __builtin_nontemporal_load(reinterpret_cast<const bf16x4_t*>(p1));
    return bf16x8_t{a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
  } else {
    return load_frag_2x8B(p0, p1);
  }
}

// fp32 softmax weights as a bf16 pair: p = hi + lo to within 2^-17, so a PV
// product of both parts keeps the weights' precision (SPLIT forms)
__device__ __forceinline__ void split_weights(const float (&p)[8], bf16x8_t& hi, bf16x8_t& lo) {
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    const uint16_t h = f2bf(p[j]);
    hi[j] = (short)h;
    lo[j] = (short)f2bf(p[j] - bf2f(h));
  }
}

// Optional output gate (ptr == nullptr: off): the finished output element is
// multiplied by sigmoid(gate), gate rows laid out like the output rows.
struct GateIn {
  const bf16_t* ptr;
  long stride;
};
__device__ __forceinline__ float gate_mul(const GateIn& gt, long row, long col, float o) {
  if (!gt.ptr) return o;
  return o / (1.f + __expf(-bf2f(gt.ptr[row * gt.stride + col])));
}

// Partition length used for a sequence: the requested split-K granule, grown
// (in 128-token steps) when the context would need more than max_parts
// partitions, so the grid baked into a captured graph always covers it.
__device__ __forceinline__ int effective_part(int ctx, int part_tokens, int max_parts) {
  int need = (ctx + max_parts - 1) / max_parts;
  need = (need + 127) & ~127;
  return need > part_tokens ? need : part_tokens;
}

}  // namespace lmx
