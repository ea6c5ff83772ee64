// K20: latent attention with a sliding window (models.mixers
// LatentAttentionMixer).  A token's cache page row is [latent c (Rp) | rotated
// key part (xp)], one row for all heads.
//
//   rope_angles    cos | sin of the step's positions (reduced in double), scaled
//   latent_prep    projection rows -> RMS-normed query latents; normed c and
//                  the rotated key part into the pages
//   latent_rotate  the rotated part of the queries that score latents
//   latent_rows    attention on latents (MFMA): a workgroup serves one query
//                  row, its heads are the MFMA columns
//   latent_any     the same for fp32 and for other sizes (fp32 arithmetic)
//   latent_gather  the cached rows a step's prompt rows see, back to back
//   latent_prefill prompt rows on keys and values expanded from those rows
#include "common.h"

namespace lmx {
namespace {

constexpr int BS = 32;   // tokens per page
constexpr float LOG2E = 1.4426950408889634f;

__global__ void __launch_bounds__(256) rope_angles_kernel(const int* __restrict__ positions,
                                                          const double* __restrict__ freqs, int T,
                                                          int n, float scale,
                                                          float* __restrict__ out) {
  const int e = blockIdx.x * 256 + threadIdx.x;
  if (e >= T * n) return;
  const int t = e / n, i = e - t * n;
  // the angle modulo one turn in double, then single precision
  const double turns = (double)positions[t] * freqs[i] * 0.15915494309189535;
  const float a = (float)((turns - floor(turns)) * 6.283185307179586);
  out[(long)t * 2 * n + i] = scale * cosf(a);
  out[(long)t * 2 * n + n + i] = scale * sinf(a);
}

// grid rows, block 256: waves 0-2 the query latent, wave 3 the cache row.
// Gains are zero in the padding, so padded columns come out zero.
template <typename T>
__global__ void __launch_bounds__(256) latent_prep_kernel(
    const T* __restrict__ p, long p_ld, int qr, int qp, const float* __restrict__ q_norm, int R,
    int Rp, const float* __restrict__ c_norm, const float* __restrict__ ang, int d,
    const int* __restrict__ slots, T* __restrict__ pages, int D, T* __restrict__ cq, float eps) {
  __shared__ float part[3];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const long row = blockIdx.x;
  const T* src = p + row * p_ld;
  if (wave == 3) {
    const int slot = slots[row];
    const T* cs = src + qp;
    float ss = 0.f;
    for (int c = lane * 8; c < Rp; c += 512) {
      float v[8];
      ldv<8>(v, cs + c);
#pragma unroll
      for (int e = 0; e < 8; ++e) ss += v[e] * v[e];
    }
    const float inv = rsqrtf(wave_sum(ss) / (float)R + eps);
    if (slot >= 0) {
      T* dst = pages + (long)slot * D;
      for (int c = lane * 8; c < Rp; c += 512) {
        float v[8], g[8];
        ldv<8>(v, cs + c);
        ldv<8>(g, c_norm + c);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] *= inv * g[e];
        stv<8>(dst + c, v);
      }
      const float* an = ang + row * d;
      const T* ks = cs + Rp;
      const int half = d / 2;
      for (int j = lane; j < D - Rp; j += 64) {
        const int i = j < half ? j : j - half;
        float o = 0.f;
        if (j < d) {
          const float a = ld1(ks + i), b = ld1(ks + half + i), cv = an[i], sv = an[half + i];
          o = j < half ? a * cv - b * sv : b * cv + a * sv;
        }
        st1(dst + Rp + j, o);
      }
    }
  } else {
    float ss = 0.f;
    for (int c = tid * 8; c < qp; c += 192 * 8) {
      float v[8];
      ldv<8>(v, src + c);
#pragma unroll
      for (int e = 0; e < 8; ++e) ss += v[e] * v[e];
    }
    ss = wave_sum(ss);
    if (lane == 0) part[wave] = ss;
  }
  __syncthreads();
  if (wave == 3) return;
  const float inv = rsqrtf((part[0] + part[1] + part[2]) / (float)qr + eps);
  for (int c = tid * 8; c < qp; c += 192 * 8) {
    float v[8], g[8];
    ldv<8>(v, src + c);
    ldv<8>(g, q_norm + c);
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] *= inv * g[e];
    stv<8>(cq + row * qp + c, v);
  }
}

// grid rows, block 256
template <typename T>
__global__ void __launch_bounds__(256) latent_rotate_kernel(const T* __restrict__ q, long q_ld,
                                                            int np, const float* __restrict__ ang,
                                                            int d, int H, int xp,
                                                            T* __restrict__ out, long o_ld, int Rp) {
  const long row = blockIdx.x;
  const float* an = ang + row * d;
  const int half = d / 2;
  for (int e = threadIdx.x; e < H * xp; e += 256) {
    const int h = e / xp, j = e - h * xp;
    const T* x = q + row * q_ld + (long)h * (np + xp) + np;
    const int i = j < half ? j : j - half;
    float o = 0.f;
    if (j < d) {
      const float a = ld1(x + i), b = ld1(x + half + i), cv = an[i], sv = an[half + i];
      o = j < half ? a * cv - b * sv : b * cv + a * sv;
    }
    st1(out + row * o_ld + (long)h * (Rp + xp) + Rp + j, o);
  }
}

// the sequence of a row (cu_q ascending)
__device__ __forceinline__ int row_seq(const int* __restrict__ cu_q, int S, int row) {
  int lo = 0, hi = S - 1;
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (cu_q[mid] <= row) lo = mid; else hi = mid - 1;
  }
  return lo;
}

// One wave per (row, head): a lane scores one key of a 64-key block, then owns
// every 64th latent channel of the weighted sum.  grid (rows, ceil(H / 4)),
// block 256, dynamic LDS 4 D floats.
template <typename T, int ND>
__global__ void __launch_bounds__(256) latent_any_kernel(
    const T* __restrict__ q, const T* __restrict__ pages, const int* __restrict__ bt, int bt_stride,
    const int* __restrict__ cu_q, int S, const int* __restrict__ positions, T* __restrict__ out,
    int H, int Rp, int D, float scale, int window) {
  extern __shared__ float sq_all[];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const long row = blockIdx.x;
  const int h = blockIdx.y * 4 + wave;
  float* sq = sq_all + wave * D;
  const bool on = h < H;
  if (on)
    for (int d = lane; d < D; d += 64) sq[d] = ld1(q + (row * H + h) * D + d);
  __syncthreads();
  if (!on) return;
  const int* tab = bt + (long)row_seq(cu_q, S, (int)row) * bt_stride;
  const int p = positions[row], j0 = max(0, p - window + 1);
  float m = -INFINITY, l = 0.f, acc[ND];
#pragma unroll
  for (int i = 0; i < ND; ++i) acc[i] = 0.f;
  for (int k0 = j0; k0 <= p; k0 += 64) {
    const int key = k0 + lane;
    float s = -INFINITY;
    if (key <= p) {
      const T* kp = pages + ((long)tab[key / BS] * BS + key % BS) * D;
      float t = 0.f;
      for (int d = 0; d < D; d += 8) {
        float x[8];
        ldv<8>(x, kp + d);
#pragma unroll
        for (int e = 0; e < 8; ++e) t += x[e] * sq[d + e];
      }
      s = t * scale;
    }
    const float mn = fmaxf(m, wave_max(s));
    const float al = expf(m - mn), w = expf(s - mn);   // exp(-inf) = 0
    l = l * al + wave_sum(w);
    m = mn;
#pragma unroll
    for (int i = 0; i < ND; ++i) acc[i] *= al;
    const int cnt = min(64, p + 1 - k0);
    for (int j = 0; j < cnt; ++j) {
      const float wj = __shfl(w, j, 64);
      const int kj = k0 + j;
      const T* vp = pages + ((long)tab[kj / BS] * BS + kj % BS) * D;
#pragma unroll
      for (int i = 0; i < ND; ++i)
        if (i * 64 < Rp) acc[i] += wj * ld1(vp + i * 64 + lane);
    }
  }
  const float inv = 1.f / l;
#pragma unroll
  for (int i = 0; i < ND; ++i)
    if (i * 64 < Rp) st1(out + (row * H + h) * Rp + i * 64 + lane, acc[i] * inv);
}

// ------------------------------------------------------ attention on latents ----
// grid (parts, head groups, rows), block 256 NG: four waves per group of 16
// heads (the MFMA columns) of one row.  Keys come in tiles of 64 (two pages)
// into a double buffer by LDS-DMA, shared by the groups; wave w of a group
// scores keys 16 w .. 16 w + 15 of the tile (S^T: keys x heads), the four agree
// on the columns' maxima, write the weights as MFMA operands (a bf16 pair, so
// they keep fp32 precision to 2^-17) and each sums its quarter of the latent's
// channels, V^T read from the same key rows with the transposing LDS read.
constexpr int TK = 64;

typedef short s16x4_t __attribute__((ext_vector_type(4)));

// Transposing LDS reads (each 16-lane group: lane i points at 4 elements of row
// i / 4, columns 4 (i % 4)..; it receives the 4 rows' elements of column i) of N
// channel tiles at byte address + OFF and, 16 rows further, + OFF + STEP: the V^T
// operands of 32 keys.  One asm block with its wait: beside LDS-DMA the
// compiler would wait for all of it before such a read.
template <int N, int OFF, int STEP>
__device__ __forceinline__ void read_vt(bf16x8_t (&f)[N], const unsigned (&at)[N]) {
  s16x4_t lo[N], hi[N];
  if constexpr (N == 1) {
    asm volatile("ds_read_b64_tr_b16 %0, %2 offset:%3\n\tds_read_b64_tr_b16 %1, %2 offset:%4\n\t"
                 "s_waitcnt lgkmcnt(0)"
                 : "=&v"(lo[0]), "=&v"(hi[0]) : "v"(at[0]), "i"(OFF), "i"(OFF + STEP) : "memory");
  } else if constexpr (N == 2) {
    asm volatile("ds_read_b64_tr_b16 %0, %4 offset:%6\n\tds_read_b64_tr_b16 %1, %4 offset:%7\n\t"
                 "ds_read_b64_tr_b16 %2, %5 offset:%6\n\tds_read_b64_tr_b16 %3, %5 offset:%7\n\t"
                 "s_waitcnt lgkmcnt(0)"
                 : "=&v"(lo[0]), "=&v"(hi[0]), "=&v"(lo[1]), "=&v"(hi[1])
                 : "v"(at[0]), "v"(at[1]), "i"(OFF), "i"(OFF + STEP) : "memory");
  } else {
    static_assert(N == 4, "1, 2 or 4 channel tiles");
    asm volatile("ds_read_b64_tr_b16 %0, %8 offset:%12\n\tds_read_b64_tr_b16 %1, %8 offset:%13\n\t"
                 "ds_read_b64_tr_b16 %2, %9 offset:%12\n\tds_read_b64_tr_b16 %3, %9 offset:%13\n\t"
                 "ds_read_b64_tr_b16 %4, %10 offset:%12\n\tds_read_b64_tr_b16 %5, %10 offset:%13\n\t"
                 "ds_read_b64_tr_b16 %6, %11 offset:%12\n\tds_read_b64_tr_b16 %7, %11 offset:%13\n\t"
                 "s_waitcnt lgkmcnt(0)"
                 : "=&v"(lo[0]), "=&v"(hi[0]), "=&v"(lo[1]), "=&v"(hi[1]), "=&v"(lo[2]),
                   "=&v"(hi[2]), "=&v"(lo[3]), "=&v"(hi[3])
                 : "v"(at[0]), "v"(at[1]), "v"(at[2]), "v"(at[3]), "i"(OFF), "i"(OFF + STEP)
                 : "memory");
  }
#pragma unroll
  for (int i = 0; i < N; ++i)
    f[i] = bf16x8_t{lo[i][0], lo[i][1], lo[i][2], lo[i][3], hi[i][0], hi[i][1], hi[i][2], hi[i][3]};
}

__device__ __forceinline__ unsigned lds_addr(const bf16_t* p) {
  return (unsigned)(uintptr_t)(__attribute__((address_space(3))) const void*)p;
}

template <int R>
__device__ __forceinline__ int lat_swz(int row) {
  constexpr int D8 = (R + 64) / 64;                   // 8-chunk groups per row
  return (D8 & 1) ? (row >> 1) & 7 : row & 7;
}

// max / sum over lanes c, c + 16, c + 32, c + 48 by VALU lane swaps
__device__ __forceinline__ float xmax(float x) {
  const unsigned u = __float_as_uint(x);
  const auto a = __builtin_amdgcn_permlane16_swap(u, u, false, false);
  x = fmaxf(__uint_as_float(a[0]), __uint_as_float(a[1]));
  const unsigned v = __float_as_uint(x);
  const auto b = __builtin_amdgcn_permlane32_swap(v, v, false, false);
  return fmaxf(__uint_as_float(b[0]), __uint_as_float(b[1]));
}
__device__ __forceinline__ float xsum(float x) {
  const unsigned u = __float_as_uint(x);
  const auto a = __builtin_amdgcn_permlane16_swap(u, u, false, false);
  x = __uint_as_float(a[0]) + __uint_as_float(a[1]);
  const unsigned v = __float_as_uint(x);
  const auto b = __builtin_amdgcn_permlane32_swap(v, v, false, false);
  return __uint_as_float(b[0]) + __uint_as_float(b[1]);
}

template <int R, int NG>
__global__ void __launch_bounds__(256 * NG, 1) latent_rows_kernel(
    const bf16_t* __restrict__ q, const bf16_t* __restrict__ pages, const int* __restrict__ bt,
    int bt_stride, const int* __restrict__ cu_q, int S, const int* __restrict__ positions,
    int num_decode, bf16_t* __restrict__ out, float* __restrict__ part_o,
    float* __restrict__ part_ml, int H, float scale, int window, int part_keys, int max_parts) {
  constexpr int D = R + 64, KS = D / 32, CH = D / 8, NT = 256 * NG;
  constexpr int DT = R / 64;                          // 16-channel tiles per wave
  extern __shared__ __attribute__((aligned(16))) char lt_smem[];
  bf16_t* const kt = reinterpret_cast<bf16_t*>(lt_smem);              // [2][TK][D]
  const int tid = threadIdx.x, lane = tid & 63, c = lane & 15, g = lane >> 4;
  const int wv = __builtin_amdgcn_readfirstlane(tid >> 6), wave = wv & 3, grp = wv >> 2;
  bf16_t* const pw = kt + 2 * TK * D + grp * 2 * 2 * 512;             // [hi, lo][2 k steps][64 x 8]
  float* const smax = reinterpret_cast<float*>(kt + 2 * TK * D + NG * 2 * 2 * 512) + grp * 64;
  const long row = blockIdx.z;
  const int part = blockIdx.x, h = (blockIdx.y * NG + grp) * 16 + c;
  const int pos = positions[row];
  const int lo = max(0, pos - window + 1);
  // the row's visible keys in parts of whole tiles
  const int base = lo / TK * TK, span = pos + 1 - base;
  int pk = max(part_keys, (span + max_parts - 1) / max_parts);
  pk = (pk + TK - 1) / TK * TK;
  const int nparts = (span + pk - 1) / pk;
  if (part >= nparts) return;
  const int b0 = base + part * pk, b1 = min(b0 + pk, pos + 1);
  const int seq = row < num_decode ? (int)row : row_seq(cu_q, S, (int)row);
  const int* tab = bt + (long)seq * bt_stride;
  const int last_page = pos / BS;

  // page ids by scalar loads: a vector load would wait behind the DMAs before it
  auto stage = [&](int t0, int buf) {
    const int pg = t0 / BS;
    const long pa = (long)tab[pg] * BS * D, pb = (long)tab[min(pg + 1, last_page)] * BS * D;
#pragma unroll
    for (int i = 0; i < TK * CH / NT; ++i) {
      const int e = i * NT + tid, r = e / CH, ch = e % CH;
      lds_dma16(pages + (r < BS ? pa : pb) + (r % BS) * D + 8 * (ch ^ lat_swz<R>(r)),
                kt + buf * TK * D + (i * NT + wv * 64) * 8);
    }
  };
  static_assert(TK * CH % NT == 0, "a tile is whole DMA instructions");

  stage(b0, 0);                       // in flight under the query loads
  bf16x8_t qf[KS];
#pragma unroll
  for (int s = 0; s < KS; ++s)
    qf[s] = load_frag16B(q + (row * H + min(h, H - 1)) * D + 32 * s + 8 * g);
  float m = -INFINITY, l = 0.f;
  f32x4_t acc[DT];
#pragma unroll
  for (int i = 0; i < DT; ++i) acc[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  const float sl = scale * LOG2E;
  int buf = 0;
  for (int t0 = b0; t0 < b1; t0 += TK, buf ^= 1) {
    dma_barrier();                    // the tile landed; every wave is done with the other buffer
    if (t0 + TK < b1) stage(t0 + TK, buf ^ 1);
    const bf16_t* tile = kt + buf * TK * D;
    // even and odd K steps: shorter MFMA chains
    f32x4_t s = {0.f, 0.f, 0.f, 0.f}, s2 = {0.f, 0.f, 0.f, 0.f};
    {
      const int r = 16 * wave + c;
      constexpr int KB = KS % 6 == 0 ? 6 : KS % 5 == 0 ? 5 : 4;   // reads in flight
      static_assert(KS % KB == 0, "whole batches");
      bf16x8_t kf[2][KB];
      auto read = [&](int b) {
#pragma unroll
        for (int j = 0; j < KB; ++j)
          kf[b & 1][j] =
              load_frag16B(tile + r * D + 8 * ((4 * (b * KB + j) + g) ^ lat_swz<R>(r)));
      };
      read(0);
#pragma unroll
      for (int b = 0; b < KS / KB; ++b) {
        if (b + 1 < KS / KB) read(b + 1);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int j = 0; j < KB; ++j) {
          f32x4_t& a = (b * KB + j) & 1 ? s2 : s;
          a = mfma16(kf[b & 1][j], qf[b * KB + j], a);
        }
        __builtin_amdgcn_sched_barrier(0);
      }
      s += s2;
    }
    float x[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int key = t0 + 16 * wave + 4 * g + r;
      x[r] = key >= lo && key < b1 ? s[r] * sl : -INFINITY;
    }
    const float wmax = xmax(fmaxf(fmaxf(x[0], x[1]), fmaxf(x[2], x[3])));
    if (g == 0) smax[wave * 16 + c] = wmax;
    lds_barrier();
    float mx = m;
#pragma unroll
    for (int w = 0; w < 4; ++w) mx = fmaxf(mx, smax[w * 16 + c]);
    const float mu = mx == -INFINITY ? 0.f : mx;
    const float al = fast_exp2(m - mu);
    const bool grew = mx > m;
    m = mx;
    float ps = 0.f;
    bf16x4_t hi, lw;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float p = fast_exp2(x[r] - mu);
      ps += p;
      const uint16_t hb = f2bf(p);
      hi[r] = (short)hb;
      lw[r] = (short)f2bf(p - bf2f(hb));
    }
    l = l * al + ps;                  // this lane's keys only; summed at the end
    // k step wave / 2, lane group g: element 4 (wave & 1) + r
    bf16_t* dst = pw + ((wave >> 1) * 64 + lane) * 8 + 4 * (wave & 1);
    *reinterpret_cast<bf16x4_t*>(dst) = hi;
    *reinterpret_cast<bf16x4_t*>(dst + 2 * 512) = lw;
    if (__ballot(grew)) {
#pragma unroll
      for (int i = 0; i < DT; ++i) acc[i] *= al;
    }
    lds_barrier();
    bf16x8_t ph[2], pl[2];
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      const bf16_t* src = pw + (ks * 64 + lane) * 8;
      ph[ks] = load_frag16B(src);
      pl[ks] = load_frag16B(src + 2 * 512);
    }
    // V^T of keys 32 ks + 4 g + .. and 16 further: row 4 g + c / 4, channel chunk
    // (rows 16 and 32 further have the same swizzle)
    constexpr int DB = DT < 4 ? DT : 4;
#pragma unroll
    for (int i0 = 0; i0 < DT; i0 += DB) {
      unsigned at[DB];
#pragma unroll
      for (int i = 0; i < DB; ++i) {
        const int r = 4 * g + (c >> 2), d0 = (wave * DT + i0 + i) * 16 + 4 * (c & 3);
        at[i] = lds_addr(tile + r * D + 8 * ((d0 >> 3) ^ lat_swz<R>(r)) + (d0 & 7));
      }
      bf16x8_t va[DB], vb[DB];
      read_vt<DB, 0, 16 * D * 2>(va, at);
#pragma unroll
      for (int i = 0; i < DB; ++i) acc[i0 + i] = mfma16(va[i], ph[0], acc[i0 + i]);
#pragma unroll
      for (int i = 0; i < DB; ++i) acc[i0 + i] = mfma16(va[i], pl[0], acc[i0 + i]);
      read_vt<DB, 32 * D * 2, 16 * D * 2>(vb, at);
#pragma unroll
      for (int i = 0; i < DB; ++i) acc[i0 + i] = mfma16(vb[i], ph[1], acc[i0 + i]);
#pragma unroll
      for (int i = 0; i < DB; ++i) acc[i0 + i] = mfma16(vb[i], pl[1], acc[i0 + i]);
    }
  }
  // denominators over the waves
  l = xsum(l);
  lds_barrier();                      // smax is free
  if (g == 0) smax[wave * 16 + c] = l;
  lds_barrier();
  if (h >= H) return;
  float L = 0.f;
#pragma unroll
  for (int w = 0; w < 4; ++w) L += smax[w * 16 + c];
  if (nparts == 1) {
    const float inv = 1.f / L;
#pragma unroll
    for (int i = 0; i < DT; ++i) {
      bf16x4_t o;
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] = (short)f2bf(acc[i][r] * inv);
      *reinterpret_cast<bf16x4_t*>(out + (row * H + h) * R + (wave * DT + i) * 16 + 4 * g) = o;
    }
  } else {
    const long idx = (row * H + h) * max_parts + part;
#pragma unroll
    for (int i = 0; i < DT; ++i)
      *reinterpret_cast<f32x4_t*>(part_o + idx * R + (wave * DT + i) * 16 + 4 * g) = acc[i];
    if (wave == 0 && g == 0) { part_ml[2 * idx] = m; part_ml[2 * idx + 1] = L; }
  }
}

// grid (H, rows), block 64: combine the parts of a row
__global__ void __launch_bounds__(64) latent_reduce_kernel(
    const float* __restrict__ part_o, const float* __restrict__ part_ml,
    const int* __restrict__ positions, bf16_t* __restrict__ out, int H, int R, int window,
    int part_keys, int max_parts) {
  const long row = blockIdx.y, h = blockIdx.x;
  const int pos = positions[row], base = max(0, pos - window + 1) / TK * TK, span = pos + 1 - base;
  int pk = max(part_keys, (span + max_parts - 1) / max_parts);
  pk = (pk + TK - 1) / TK * TK;
  const int nparts = (span + pk - 1) / pk;
  if (nparts == 1) return;
  const long idx = (row * H + h) * max_parts;
  float M = -INFINITY;
  for (int p = 0; p < nparts; ++p) M = fmaxf(M, part_ml[2 * (idx + p)]);
  for (int d = threadIdx.x * 4; d < R; d += 256) {
    float L = 0.f;
    f32x4_t o = {0.f, 0.f, 0.f, 0.f};
    for (int p = 0; p < nparts; ++p) {
      const float mp = part_ml[2 * (idx + p)], f = mp == -INFINITY ? 0.f : fast_exp2(mp - M);
      L += f * part_ml[2 * (idx + p) + 1];
      o += f * *reinterpret_cast<const f32x4_t*>(part_o + (idx + p) * R + d);
    }
    bf16x4_t r;
#pragma unroll
    for (int e = 0; e < 4; ++e) r[e] = (short)f2bf(o[e] / L);
    *reinterpret_cast<bf16x4_t*>(out + (row * H + h) * R + d) = r;
  }
}

// ------------------------------------------------------------- prompt rows ----
// seqs[s] = (first gathered row, first position) of sequence s, S + 1 entries
__device__ __forceinline__ int gathered_seq(const int* __restrict__ seqs, int S, int row) {
  int lo = 0, hi = S - 1;
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (seqs[2 * mid] <= row) lo = mid; else hi = mid - 1;
  }
  return lo;
}

// grid ceil(n / 4), block 256: one wave per row
__global__ void __launch_bounds__(256) latent_gather_kernel(const bf16_t* __restrict__ pages,
                                                            const int* __restrict__ bt,
                                                            int bt_stride,
                                                            const int* __restrict__ seqs, int S,
                                                            int n, int D, bf16_t* __restrict__ out) {
  const int row = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (row >= n) return;
  const int s = gathered_seq(seqs, S, row), pos = row - seqs[2 * s] + seqs[2 * s + 1];
  const bf16_t* src = pages + ((long)bt[(long)s * bt_stride + pos / BS] * BS + pos % BS) * D;
  for (int c = lane * 8; c < D; c += 512)
    *reinterpret_cast<u16x8*>(out + (long)row * D + c) = *reinterpret_cast<const u16x8*>(src + c);
}

// 8 elements j0.. of a rotated part x [d of 64] by the angles an [d] (cos | sin)
__device__ __forceinline__ bf16x8_t rotated_frag(const bf16_t* __restrict__ x,
                                                 const float* __restrict__ an, int d, int j0) {
  const int half = d / 2;
  bf16x8_t o = {0, 0, 0, 0, 0, 0, 0, 0};
  if (j0 >= d) return o;
  if (half % 8 == 0) {
    const bool up = j0 >= half;
    const int i0 = up ? j0 - half : j0;
    const bf16x8_t lo = load_frag16B(x + i0), hi = load_frag16B(x + half + i0);
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float a = bf2f((uint16_t)lo[e]), b = bf2f((uint16_t)hi[e]);
      const float cv = an[i0 + e], sv = an[half + i0 + e];
      o[e] = (short)f2bf(up ? b * cv + a * sv : a * cv - b * sv);
    }
    return o;
  }
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    const int j = j0 + e, i = j < half ? j : j - half;
    if (j < d) {
      const float a = bf2f(x[i]), b = bf2f(x[half + i]), cv = an[i], sv = an[half + i];
      o[e] = (short)f2bf(j < half ? a * cv - b * sv : b * cv + a * sv);
    }
  }
  return o;
}

template <int CH>
__device__ __forceinline__ int pre_swz(int row) {
  return CH % 16 == 0 ? row & 15 : (row >> 1) & 7;
}

// One head of one 128-query tile per workgroup; a wave owns NG groups of 16
// queries (MFMA columns).  Keys W_uk c | rotated part and values W_uv c come in
// 64-key tiles by LDS-DMA, double-buffered; S^T leaves the weights where the
// PV product reads them (permuted keys, as in attention.hip), V^T comes from
// the value rows with the transposing LDS read.  Weights enter PV as a bf16
// pair.  grid tiles x heads, block 256.
struct LatentPre {
  const bf16_t* q;        // rows [H][NP + 64], not rotated
  const bf16_t* kv;       // gathered rows [H][NP + VP]
  const bf16_t* lat;      // gathered rows [D], rotated key part from Rp
  const float* ang;       // [rows][d]
  const int *seqs, *tiles, *cu_q, *ctx;
  const bf16_t* gate;     // rows [H][VP]
  bf16_t* out;            // rows [H][VP]
  long q_ld, gate_ld, out_ld;
  int ntiles, H, D, Rp, d, window;
  float scale;
};

template <int NP, int VP>
__global__ void __launch_bounds__(256, 2) latent_prefill_kernel(LatentPre p) {
  constexpr int NG = 2, KD = NP + 64, KS = KD / 32, KC = KD / 8, VC = VP / 8, VT = VP / 16;
  constexpr int KN = TK * KC / 256, VN = TK * VC / 256;   // DMA instructions per tile
  extern __shared__ __attribute__((aligned(16))) char lp_smem[];
  bf16_t* const sk = reinterpret_cast<bf16_t*>(lp_smem);            // [2][TK][KD]
  bf16_t* const sv = sk + 2 * TK * KD;                              // [2][TK][VP]
  const int tid = threadIdx.x, lane = tid & 63, c = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  // a head's tiles are consecutive on one XCD: they share its keys in L2; the
  // list is walked backwards (long key walks first)
  const int lin = xcd_remap(blockIdx.x, gridDim.x);
  const int h = lin / p.ntiles, tile = p.ntiles - 1 - lin % p.ntiles;
  const int s = p.tiles[2 * tile], q0 = p.tiles[2 * tile + 1];
  const int qbeg = p.cu_q[s], qlen = p.cu_q[s + 1] - qbeg, p0 = p.ctx[s] - qlen;
  const int k0 = p.seqs[2 * s + 1];                       // first gathered position
  const long krow = (long)p.seqs[2 * s] - k0;             // gathered row of position 0
  const int wq1 = min(q0 + 128, qlen);                    // one past the tile's last query
  const int kmax = p0 + wq1 - 1;
  const int t_lo = k0 + (max(p0 + q0 - p.window + 1, k0) - k0) / TK * TK;

  const bf16_t* src[KN + VN];
  int srow[KN + VN];
  long sld[KN + VN];
  const long kvld = (long)p.H * (NP + VP);
#pragma unroll
  for (int i = 0; i < KN; ++i) {
    const int e = i * 256 + tid, r = e / KC, ch = (e % KC) ^ pre_swz<KC>(r);
    srow[i] = r;
    const bool kr = ch >= NP / 8;
    src[i] = kr ? p.lat + p.Rp + 8 * (ch - NP / 8) : p.kv + (long)h * (NP + VP) + 8 * ch;
    sld[i] = kr ? p.D : kvld;
  }
#pragma unroll
  for (int i = 0; i < VN; ++i) {
    const int e = i * 256 + tid, r = e / VC, ch = (e % VC) ^ pre_swz<VC>(r);
    srow[KN + i] = r;
    src[KN + i] = p.kv + (long)h * (NP + VP) + NP + 8 * ch;
    sld[KN + i] = kvld;
  }
  auto stage = [&](int t0, int buf) {
#pragma unroll
    for (int i = 0; i < KN + VN; ++i) {
      bf16_t* dst = i < KN ? sk + buf * TK * KD + (i * 256 + wave * 64) * 8
                           : sv + buf * TK * VP + ((i - KN) * 256 + wave * 64) * 8;
      lds_dma16(src[i] + (krow + min(t0 + srow[i], kmax)) * sld[i], dst);
    }
  };
  stage(t_lo, 0);

  int pos[NG];
  bf16x8_t qf[NG][KS];
#pragma unroll
  for (int n = 0; n < NG; ++n) {
    const int qi = q0 + (wave * NG + n) * 16 + c;
    pos[n] = p0 + qi;
    const long row = qbeg + min(qi, qlen - 1);
    const bf16_t* qr = p.q + row * p.q_ld + (long)h * KD;
#pragma unroll
    for (int ks = 0; ks < NP / 32; ++ks) qf[n][ks] = load_frag16B(qr + 32 * ks + 8 * g);
#pragma unroll
    for (int ks = 0; ks < 2; ++ks)
      qf[n][NP / 32 + ks] = rotated_frag(qr + NP, p.ang + row * p.d, p.d, 32 * ks + 8 * g);
  }
  const int w0 = q0 + wave * NG * 16;                     // the wave's first query
  const bool idle = w0 >= qlen;
  const int whi = p0 + min(w0 + NG * 16, qlen) - 1;       // its last query's position
  const int wlo = p0 + w0 - p.window + 1;                 // first key any of them sees
  float m[NG], l[NG];
  f32x4_t acc[NG][VT];
#pragma unroll
  for (int n = 0; n < NG; ++n) {
    m[n] = -INFINITY;
    l[n] = 0.f;
#pragma unroll
    for (int i = 0; i < VT; ++i) acc[n][i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  }
  const float sl = p.scale * LOG2E;
  int buf = 0;
  for (int t0 = t_lo; t0 <= kmax; t0 += TK, buf ^= 1) {
    dma_barrier();                    // the tile landed; every wave is done with the other buffer
    if (t0 + TK <= kmax) stage(t0 + TK, buf ^ 1);
    if (idle || t0 > whi || t0 + TK <= wlo) continue;
    const bf16_t* kt = sk + buf * TK * KD;
    const bf16_t* vt = sv + buf * TK * VP;
    f32x4_t sc[NG][4];
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) {
      const int r = 16 * kb + c;
#pragma unroll
      for (int n = 0; n < NG; ++n) sc[n][kb] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const bf16x8_t kf = load_frag16B(kt + r * KD + 8 * ((4 * ks + g) ^ pre_swz<KC>(r)));
#pragma unroll
        for (int n = 0; n < NG; ++n) sc[n][kb] = mfma16(kf, qf[n][ks], sc[n][kb]);
      }
    }
    // every key of the tile visible to every query of the wave: no mask
    const bool mask = t0 + TK - 1 > p0 + w0 || t0 < whi - p.window + 1;
    bf16x8_t ph[NG][2], pl[NG][2];
    float al[NG];
    bool grew = false;
#pragma unroll
    for (int n = 0; n < NG; ++n) {
      float mx = -INFINITY;
      if (mask) {
#pragma unroll
        for (int kb = 0; kb < 4; ++kb)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int key = t0 + 16 * kb + 4 * g + r;
            if (key > pos[n] || key <= pos[n] - p.window) sc[n][kb][r] = -INFINITY;
          }
      }
#pragma unroll
      for (int kb = 0; kb < 4; ++kb)
        mx = fmaxf(mx, fmaxf(fmaxf(sc[n][kb][0], sc[n][kb][1]), fmaxf(sc[n][kb][2], sc[n][kb][3])));
      mx = xmax(mx) * sl;
      const float mn = fmaxf(m[n], mx);
      const float mu = mn == -INFINITY ? 0.f : mn;
      al[n] = fast_exp2(m[n] - mu);
      grew |= mn > m[n];
      m[n] = mn;
      float ps = 0.f;
#pragma unroll
      for (int kb = 0; kb < 4; ++kb)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float w = fast_exp2(sc[n][kb][r] * sl - mu);
          ps += w;
          const uint16_t hb = f2bf(w);
          ph[n][kb >> 1][4 * (kb & 1) + r] = (short)hb;
          pl[n][kb >> 1][4 * (kb & 1) + r] = (short)f2bf(w - bf2f(hb));
        }
      l[n] = l[n] * al[n] + ps;       // this lane's keys only; summed at the end
    }
    if (__ballot(grew)) {
#pragma unroll
      for (int n = 0; n < NG; ++n)
#pragma unroll
        for (int i = 0; i < VT; ++i) acc[n][i] *= al[n];
    }
#pragma unroll
    for (int i0 = 0; i0 < VT; i0 += 4) {
      unsigned at[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int r = 4 * g + (c >> 2), d0 = 16 * (i0 + i) + 4 * (c & 3);
        at[i] = lds_addr(vt + r * VP + 8 * ((d0 >> 3) ^ pre_swz<VC>(r)) + (d0 & 7));
      }
      bf16x8_t vf[4];
      read_vt<4, 0, 16 * VP * 2>(vf, at);
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int n = 0; n < NG; ++n) acc[n][i0 + i] = mfma16(vf[i], ph[n][0], acc[n][i0 + i]);
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int n = 0; n < NG; ++n) acc[n][i0 + i] = mfma16(vf[i], pl[n][0], acc[n][i0 + i]);
      read_vt<4, 32 * VP * 2, 16 * VP * 2>(vf, at);
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int n = 0; n < NG; ++n) acc[n][i0 + i] = mfma16(vf[i], ph[n][1], acc[n][i0 + i]);
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int n = 0; n < NG; ++n) acc[n][i0 + i] = mfma16(vf[i], pl[n][1], acc[n][i0 + i]);
    }
  }
#pragma unroll
  for (int n = 0; n < NG; ++n) {
    const float L = xsum(l[n]);
    const int qi = q0 + (wave * NG + n) * 16 + c;
    if (qi >= qlen) continue;
    const float inv = 1.f / L;
    const long row = qbeg + qi;
#pragma unroll
    for (int i = 0; i < VT; ++i) {
      const long col = (long)h * VP + 16 * i + 4 * g;
      const bf16x4_t gt = *reinterpret_cast<const bf16x4_t*>(p.gate + row * p.gate_ld + col);
      bf16x4_t o;
#pragma unroll
      for (int r = 0; r < 4; ++r)
        o[r] = (short)f2bf(acc[n][i][r] * inv / (1.f + __expf(-bf2f((uint16_t)gt[r]))));
      *reinterpret_cast<bf16x4_t*>(p.out + row * p.out_ld + col) = o;
    }
  }
}

}  // namespace

int rope_angles(const int* positions, const double* freqs, int T, int n, float scale, float* out,
                hipStream_t stream) {
  if (T <= 0 || n <= 0) return 0;
  rope_angles_kernel<<<dim3((T * n + 255) / 256), dim3(256), 0, stream>>>(positions, freqs, T, n, scale,
                                                                     out);
  return (int)hipGetLastError();
}

int latent_prep(const void* p, long p_ld, int T, int qr, int qp, const float* q_norm, int R, int Rp,
                const float* c_norm, const float* ang, int d, const int* slots, void* pages,
                int block_size, int D, void* cq, float eps, int is_bf16, hipStream_t stream) {
  if (T <= 0) return 0;
  if (block_size != BS || qp % 8 || Rp % 8 || D % 8 || qr < 1 || qr > qp || R < 1 || R > Rp ||
      d < 2 || d % 2 || d > D - Rp || p_ld % 8)
    return -1;
  if (is_bf16)
    latent_prep_kernel<bf16_t><<<dim3(T), dim3(256), 0, stream>>>(
        (const bf16_t*)p, p_ld, qr, qp, q_norm, R, Rp, c_norm, ang, d, slots, (bf16_t*)pages, D,
        (bf16_t*)cq, eps);
  else
    latent_prep_kernel<float><<<dim3(T), dim3(256), 0, stream>>>(
        (const float*)p, p_ld, qr, qp, q_norm, R, Rp, c_norm, ang, d, slots, (float*)pages, D,
        (float*)cq, eps);
  return (int)hipGetLastError();
}

int latent_rotate(const void* q, long q_ld, int np, const float* ang, int d, int T, int H, int xp,
                  void* out, long o_ld, int Rp, int is_bf16, hipStream_t stream) {
  if (T <= 0) return 0;
  if (d < 2 || d % 2 || d > xp || H < 1) return -1;
  if (is_bf16)
    latent_rotate_kernel<bf16_t><<<dim3(T), dim3(256), 0, stream>>>(
        (const bf16_t*)q, q_ld, np, ang, d, H, xp, (bf16_t*)out, o_ld, Rp);
  else
    latent_rotate_kernel<float><<<dim3(T), dim3(256), 0, stream>>>(
        (const float*)q, q_ld, np, ang, d, H, xp, (float*)out, o_ld, Rp);
  return (int)hipGetLastError();
}

int latent_any(const void* q, const void* pages, const int* bt, int bt_stride, const int* cu_q,
               int S, const int* positions, int rows, void* out, int H, int Rp, int D, float scale,
               int window, int is_bf16, hipStream_t stream) {
  if (rows <= 0) return 0;
  if (S < 1 || H < 1 || Rp % 64 || D % 8 || Rp >= D || window < 1 || D > 4096) return -1;
  const dim3 grid(rows, (H + 3) / 4);
  const size_t smem = 4 * D * sizeof(float);
#define LMX_LA(T, ND)                                                                          \
  latent_any_kernel<T, ND><<<grid, dim3(256), smem, stream>>>(                                 \
      (const T*)q, (const T*)pages, bt, bt_stride, cu_q, S, positions, (T*)out, H, Rp, D,      \
      scale, window)
#define LMX_LAN(T)                                                                             \
  if (Rp <= 128) LMX_LA(T, 2); else if (Rp <= 256) LMX_LA(T, 4);                               \
  else if (Rp <= 512) LMX_LA(T, 8); else if (Rp <= 1024) LMX_LA(T, 16); else return -2;
  if (is_bf16) { LMX_LAN(bf16_t) } else { LMX_LAN(float) }
#undef LMX_LAN
#undef LMX_LA
  return (int)hipGetLastError();
}

// rows before num_decode: row i is sequence i's first row.  part_o / part_ml:
// [rows][H][max_parts][Rp] / [..][2] (max_parts > 1)
int latent_rows(const void* q, const void* pages, const int* bt, int bt_stride, const int* cu_q,
                int S, const int* positions, int rows, int num_decode, void* out, float* part_o,
                float* part_ml, int H, int Rp, int D, float scale, int window, int part_keys,
                int max_parts, hipStream_t stream) {
  if (rows <= 0) return 0;
  if (S < 1 || H < 1 || window < 1 || D != Rp + 64 || part_keys < TK || max_parts < 1 ||
      (max_parts > 1 && (!part_o || !part_ml)) || rows > 65535)
    return -1;
#define LMX_LR(R, NG)                                                                          \
  {                                                                                            \
    constexpr int smem = 2 * TK * (R + 64) * 2 + 2 * 2 * NG * 512 * 2 + 4 * NG * 16 * 4;       \
    static bool attr = false;                                                                  \
    if (smem > 65536 && !attr) {                                                               \
      (void)hipFuncSetAttribute((const void*)latent_rows_kernel<R, NG>,                        \
                                hipFuncAttributeMaxDynamicSharedMemorySize, smem);             \
      attr = true;                                                                             \
    }                                                                                          \
    latent_rows_kernel<R, NG>                                                                  \
        <<<dim3(max_parts, (H + 16 * NG - 1) / (16 * NG), rows), dim3(256 * NG), smem, stream>>>(   \
            (const bf16_t*)q, (const bf16_t*)pages, bt, bt_stride, cu_q, S, positions,         \
            num_decode, (bf16_t*)out, part_o, part_ml, H, scale, window, part_keys, max_parts); \
  }
#define LMX_LRN(R) if (H <= 16) LMX_LR(R, 1) else LMX_LR(R, 2)
  if (Rp == 64) { LMX_LRN(64) } else if (Rp == 128) { LMX_LRN(128) }
  else if (Rp == 256) { LMX_LRN(256) } else if (Rp == 512) { LMX_LRN(512) }
  else return -2;
#undef LMX_LRN
#undef LMX_LR
  if (max_parts > 1)
    latent_reduce_kernel<<<dim3(H, rows), dim3(64), 0, stream>>>(
        part_o, part_ml, positions, (bf16_t*)out, H, Rp, window, part_keys, max_parts);
  return (int)hipGetLastError();
}

int latent_gather(const void* pages, const int* bt, int bt_stride, const int* seqs, int S, int n,
                  int D, void* out, hipStream_t stream) {
  if (n <= 0) return 0;
  if (S < 1 || D % 8) return -1;
  latent_gather_kernel<<<dim3((n + 3) / 4), dim3(256), 0, stream>>>(
      (const bf16_t*)pages, bt, bt_stride, seqs, S, n, D, (bf16_t*)out);
  return (int)hipGetLastError();
}

int latent_prefill(const void* q, long q_ld, const void* kv, const void* lat, const float* ang,
                   const int* seqs, const int* tiles, int ntiles, const int* cu_q, const int* ctx,
                   const void* gate, long gate_ld, void* out, long out_ld, int H, int NP, int VP,
                   int D, int Rp, int d, float scale, int window, hipStream_t stream) {
  if (ntiles <= 0) return 0;
  if (H < 1 || D != Rp + 64 || D % 8 || d < 2 || d % 2 || d > 64 || window < 1 || q_ld % 8 ||
      gate_ld % 4 || out_ld % 4)
    return -1;
  const LatentPre p{(const bf16_t*)q, (const bf16_t*)kv, (const bf16_t*)lat, ang, seqs, tiles, cu_q,
                    ctx, (const bf16_t*)gate, (bf16_t*)out, q_ld, gate_ld, out_ld, ntiles, H, D, Rp,
                    d, window, scale};
#define LMX_LP(NPV, VPV)                                                                       \
  {                                                                                            \
    constexpr int smem = 2 * TK * (NPV + 64 + VPV) * 2;                                        \
    static bool attr = false;                                                                  \
    if (smem > 65536 && !attr) {                                                               \
      (void)hipFuncSetAttribute((const void*)latent_prefill_kernel<NPV, VPV>,                  \
                                hipFuncAttributeMaxDynamicSharedMemorySize, smem);             \
      attr = true;                                                                             \
    }                                                                                          \
    latent_prefill_kernel<NPV, VPV><<<dim3(ntiles * H), dim3(256), smem, stream>>>(p);         \
  }
  if (NP == 64 && VP == 64) LMX_LP(64, 64)
  else if (NP == 64 && VP == 128) LMX_LP(64, 128)
  else if (NP == 128 && VP == 64) LMX_LP(128, 64)
  else if (NP == 128 && VP == 128) LMX_LP(128, 128)
  else return -2;
#undef LMX_LP
  return (int)hipGetLastError();
}

}  // namespace lmx
