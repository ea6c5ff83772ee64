// K19: gated linear recurrence over time, per channel, with block-diagonal
// gates of the input (see ops.rglru):
//
//   r, i = sigmoid(G u + b),  a = exp(log_a r),
//   S <- a S + sqrt(1 - a^2) i u,   out = S gelu(y + y_b)
//
// The recurrence and everything that enters it is fp32; u, y, out are bf16 (or
// fp32) rows.
//
//   rglru_chunk_kernel  prompt rows: a workgroup walks one row segment of a
//       sequence in 64-token chunks for 64 channels.  A wave owns 16 channels:
//       both gates' weights stay in registers (MFMA fragments of the packed
//       layout), the chunk's u rows of the gate block come by LDS-DMA one
//       chunk ahead.  The accumulators leave a lane with 4 consecutive tokens
//       of one channel per 16-token tile, so the scan runs in registers: 4
//       tokens in the lane, then (a, b) pairs across the 4 lane groups.
//       Sequences cut into segments take three passes: each segment's (prod a,
//       end state from zero), then the same walk from the chained start.
//   rglru_rows_kernel   decode rows: 16 sequences x 16 channels per wave
//   rglru_scan_kernel   any sizes: fp32 gates computed before, one thread per
//       (sequence, channel)
#include "common.h"

namespace lmx {
namespace {

constexpr int TC = 64;           // tokens per chunk
constexpr int CT = 64;           // channels per workgroup (ops RGLRU_TILE)
constexpr float L2E = 1.4426950408889634f;

struct RglruArgs {
  const void *u, *y;
  long y_ld;
  const float *y_b, *g_b, *log_a;
  void* out;
  float* state;                  // [slots][C]
  const int *cu_q, *ctx, *slots;
  int C, bp;
  const bf16_t* w;               // packed [blocks][2 bp / 16][bp / 32][64][8]
};

__device__ __forceinline__ float fast_sigmoid(float x) {
  return __builtin_amdgcn_rcpf(1.f + fast_exp2(-L2E * x));
}

// y / 2 (1 + tanh(k (y + 0.044715 y^3))) = y sigmoid(2 k (..))
__device__ __forceinline__ float fast_gelu(float y) {
  return y * fast_sigmoid(1.5957691216057308f * (y + 0.044715f * y * y * y));
}

// a = e^x and sqrt(1 - e^2x) for x <= 0; near 0 the difference is a series
__device__ __forceinline__ void decay_pair(float x, float& a, float& s) {
  a = fast_exp2(L2E * x);
  const float z = 2.f * x;
  const float near = -z * (1.f + z * (0.5f + z * (1.f / 6.f + z * (1.f / 24.f))));
  s = __builtin_amdgcn_sqrtf(z > -0.05f ? near : 1.f - a * a);
}

// ------------------------------------------------------------- prompt rows ----
// grid (segments, channel tiles), block 256.
// PASS 0: one pass; 1: segment ends to ws; 2: from the chained starts.
template <int KS, int PASS>
__global__ void __launch_bounds__(256, 2) rglru_chunk_kernel(RglruArgs p, int seq0,
                                                             const int* __restrict__ segs,
                                                             int nsegs,
                                                             const int* __restrict__ first,
                                                             float* __restrict__ ws) {
  constexpr int KW = KS == 1 ? 64 : KS * 32;            // staged columns
  constexpr int UCH = KW / 8;                           // 16-B chunks per row
  extern __shared__ __attribute__((aligned(16))) char rg_smem[];
  bf16_t* const su = reinterpret_cast<bf16_t*>(rg_smem);            // [2][TC][KW]
  bf16_t* const sy = su + 2 * TC * KW;                              // [2][TC][CT]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, q = lane >> 4;
  const int seg = blockIdx.x, ct = blockIdx.y;
  const int seq = segs[4 * seg], r0 = segs[4 * seg + 1], r1 = segs[4 * seg + 2];
  const bool last = segs[4 * seg + 3];
  const int slot = p.slots[seq];
  if (slot < 0) return;
  const int row0 = p.cu_q[seq], n = p.cu_q[seq + 1] - row0;
  const bool fresh = p.ctx[seq] == n;
  const int cb = ct * CT + wave * 16;                   // this wave's first channel
  const bool on = cb < p.C;
  const int ch = on ? cb + c : 0;                       // this lane's channel
  const int col0 = ct * CT / KW * KW;                   // first staged column
  const int blk = (on ? cb : 0) / p.bp, in_blk = (on ? cb : 0) - blk * p.bp;
  const int kcol = (on ? blk * p.bp - col0 : 0);        // the gate block inside the staged columns

  bf16x8_t wr[KS], wi[KS];
  {
    const bf16_t* w = p.w + ((long)blk * (2 * p.bp / 16) + in_blk / 16) * KS * 512 + lane * 8;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      wr[s] = load_frag16B(w + s * 512);
      wi[s] = load_frag16B(w + (long)(p.bp / 16) * KS * 512 + s * 512);
    }
  }
  const float br = p.g_b[ch], bi = p.g_b[p.C + ch], la = p.log_a[ch], yb = p.y_b[ch];
  const bf16_t* ub = (const bf16_t*)p.u + (long)row0 * p.C;
  const bf16_t* ybase = (const bf16_t*)p.y + (long)row0 * p.y_ld;

  auto stage = [&](int t0, int buf) {
#pragma unroll
    for (int i = 0; i < TC * UCH / 256; ++i) {
      const int e = i * 256 + tid, row = e / UCH, chn = (e % UCH) ^ (row & 7);
      const int col = min(col0 + 8 * chn, p.C - 8);
      lds_dma16(ub + (long)min(t0 + row, r1 - 1) * p.C + col,
                su + buf * TC * KW + (i * 256 + wave * 64) * 8);
    }
    if constexpr (PASS != 1) {
#pragma unroll
      for (int i = 0; i < TC * CT / 8 / 256; ++i) {
        const int e = i * 256 + tid, row = e >> 3;
        const int col = min(ct * CT + 8 * (e & 7), p.C - 8);
        lds_dma16(ybase + (long)min(t0 + row, r1 - 1) * p.y_ld + col,
                  sy + buf * TC * CT + (i * 256 + wave * 64) * 8);
      }
    }
  };

  // ws: [3][nsegs][C]: prod a, end state from zero, the sequence's start state
  float S = 0.f, A = 1.f;
  if constexpr (PASS == 0) {
    S = fresh ? 0.f : p.state[(long)slot * p.C + ch];
  } else if constexpr (PASS == 1) {
    if (r0 == 0 && on && q == 0)
      ws[(2L * nsegs + seg) * p.C + ch] = fresh ? 0.f : p.state[(long)slot * p.C + ch];
  } else {
    const int s0 = first[seq - seq0];
    S = ws[(2L * nsegs + s0) * p.C + ch];
    for (int s = s0; s < seg; ++s)
      S = ws[(long)s * p.C + ch] * S + ws[((long)nsegs + s) * p.C + ch];
  }

  stage(r0, 0);
  int buf = 0;
  for (int t0 = r0; t0 < r1; t0 += TC, buf ^= 1) {
    dma_barrier();                       // chunk landed; every wave is done with the other buffer
    if (t0 + TC < r1) stage(t0 + TC, buf ^ 1);
    const bf16_t* uc = su + buf * TC * KW;
    const bf16_t* yc = sy + buf * TC * CT;
#pragma unroll
    for (int mt = 0; mt < TC / 16; ++mt) {
      if (t0 + 16 * mt >= r1) break;
      f32x4_t zr = {br, br, br, br}, zi = {bi, bi, bi, bi};
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        const int row = 16 * mt + c;
        const bf16x8_t x =
            load_frag16B(uc + row * KW + 8 * ((kcol / 8 + 4 * s + q) ^ (row & 7)));
        zr = mfma16(x, wr[s], zr);
        zi = mfma16(x, wi[s], zi);
      }
      // tokens 16 mt + 4 q + j of channel ch
      float a[4], b[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int row = 16 * mt + 4 * q + j, col = (on ? ch : col0) - col0;
        const float u = bf2f(uc[row * KW + (((col >> 3) ^ (row & 7)) << 3) + (col & 7)]);
        float s;
        decay_pair(la * fast_sigmoid(zr[j]), a[j], s);
        b[j] = s * fast_sigmoid(zi[j]) * u;
        if (t0 + row >= r1) { a[j] = 1.f; b[j] = 0.f; }
      }
      // inclusive pairs inside the lane, then across the 4 lane groups
      float pa = a[0], pb = b[0];
#pragma unroll
      for (int j = 1; j < 4; ++j) {
        pb = a[j] * pb + b[j];
        pa = a[j] * pa;
      }
      float xa = __shfl_up(pa, 16, 64), xb = __shfl_up(pb, 16, 64);
      float ia = pa, ib = pb;
      if (q >= 1) { ib = pa * xb + pb; ia = pa * xa; }
      xa = __shfl_up(ia, 32, 64);
      xb = __shfl_up(ib, 32, 64);
      if (q >= 2) { ib = ia * xb + ib; ia = ia * xa; }
      float ea = __shfl_up(ia, 16, 64), eb = __shfl_up(ib, 16, 64);
      if (q == 0) { ea = 1.f; eb = 0.f; }
      float s = ea * S + eb;
      const float ta = __shfl(ia, 48 + c, 64), tb = __shfl(ib, 48 + c, 64);
      if constexpr (PASS != 1) {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          s = a[j] * s + b[j];
          const int row = 16 * mt + 4 * q + j;
          const float g = fast_gelu(bf2f(yc[row * CT + wave * 16 + c]) + yb);
          if (on && t0 + row < r1)
            ((bf16_t*)p.out)[(long)(row0 + t0 + row) * p.C + ch] = f2bf(s * g);
        }
      }
      S = ta * S + tb;
      A *= ta;
    }
  }
  if (!on || q != 0) return;
  if constexpr (PASS == 1) {
    ws[(long)seg * p.C + ch] = A;
    ws[((long)nsegs + seg) * p.C + ch] = S;
  } else if (last) {
    p.state[(long)slot * p.C + ch] = S;
  }
}

// ------------------------------------------------------------- decode rows ----
// grid (channel tiles, ceil(rows / 16)), block 256: row i is sequence i's
template <int KS>
__global__ void __launch_bounds__(256) rglru_rows_kernel(RglruArgs p, int rows) {
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, q = lane >> 4;
  const int cb = blockIdx.x * CT + wave * 16, t0 = blockIdx.y * 16;
  if (cb >= p.C) return;
  const int ch = cb + c, blk = cb / p.bp, in_blk = cb - blk * p.bp;
  const bf16_t* w = p.w + ((long)blk * (2 * p.bp / 16) + in_blk / 16) * KS * 512 + lane * 8;
  const bf16_t* ur = (const bf16_t*)p.u + (long)min(t0 + c, rows - 1) * p.C + blk * p.bp;
  // everything the epilogue needs, in flight under the products
  int slot[4];
  bool fresh[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int t = t0 + 4 * q + j;
    slot[j] = t < rows ? p.slots[t] : -1;
    fresh[j] = t < rows && p.ctx[t] == 1;
  }
  const float br = p.g_b[ch], bi = p.g_b[p.C + ch], la = p.log_a[ch], yb = p.y_b[ch];
  bf16x8_t x[KS], wr[KS], wi[KS];
#pragma unroll
  for (int s = 0; s < KS; ++s) {
    x[s] = load_frag16B(ur + 32 * s + 8 * q);
    wr[s] = load_frag16B(w + s * 512);
    wi[s] = load_frag16B(w + (long)(p.bp / 16) * KS * 512 + s * 512);
  }
  float S0[4], u[4], y[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const long t = min(t0 + 4 * q + j, rows - 1);
    S0[j] = p.state[(long)max(slot[j], 0) * p.C + ch];
    u[j] = bf2f(((const bf16_t*)p.u)[t * p.C + ch]);
    y[j] = bf2f(((const bf16_t*)p.y)[t * p.y_ld + ch]);
  }
  f32x4_t zr = {br, br, br, br}, zi = {bi, bi, bi, bi};
#pragma unroll
  for (int s = 0; s < KS; ++s) {
    zr = mfma16(x[s], wr[s], zr);
    zi = mfma16(x[s], wi[s], zi);
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    if (slot[j] < 0) continue;
    float a, s;
    decay_pair(la * fast_sigmoid(zr[j]), a, s);
    const float S = (fresh[j] ? 0.f : a * S0[j]) + s * fast_sigmoid(zi[j]) * u[j];
    p.state[(long)slot[j] * p.C + ch] = S;
    ((bf16_t*)p.out)[(long)(t0 + 4 * q + j) * p.C + ch] = f2bf(S * fast_gelu(y[j] + yb));
  }
}

// ---------------------------------------------------------------- any sizes ----
// z: fp32 gate products [T][blocks][2][bp]; grid (sequences, ceil(C / 64)), block 64
template <typename T>
__global__ void __launch_bounds__(64) rglru_scan_kernel(RglruArgs p, const float* __restrict__ z) {
  const int seq = blockIdx.x, ch = blockIdx.y * 64 + threadIdx.x;
  const int slot = p.slots[seq];
  if (ch >= p.C || slot < 0) return;
  const int row0 = p.cu_q[seq], n = p.cu_q[seq + 1] - row0;
  float* st = p.state + (long)slot * p.C + ch;
  float S = p.ctx[seq] == n ? 0.f : *st;
  const int blk = ch / p.bp;
  const long zc = (long)blk * 2 * p.bp + (ch - blk * p.bp);
  const float br = p.g_b[ch], bi = p.g_b[p.C + ch], la = p.log_a[ch], yb = p.y_b[ch];
#pragma unroll 4
  for (int t = 0; t < n; ++t) {
    const long row = row0 + t;
    const float r = 1.f / (1.f + expf(-(z[row * 2 * p.C + zc] + br)));
    const float i = 1.f / (1.f + expf(-(z[row * 2 * p.C + zc + p.bp] + bi)));
    const float x = la * r;
    S = expf(x) * S + sqrtf(-expm1f(2.f * x)) * i * ld1((const T*)p.u + row * p.C + ch);
    const float y = ld1((const T*)p.y + row * p.y_ld + ch) + yb;
    const float g = 0.5f * y * (1.f + tanhf(0.7978845608028654f * (y + 0.044715f * y * y * y)));
    st1((T*)p.out + row * p.C + ch, S * g);
  }
  *st = S;
}

bool rglru_ok(const RglruArgs& p, bool packed) {
  if (p.C < 1 || p.bp < 1 || p.C % p.bp) return false;
  if (!packed) return true;
  const int ks = p.bp / 32;
  return p.bp % 32 == 0 && p.C % 16 == 0 && (ks == 1 || ks == 2 || ks == 4 || ks == 8 || ks == 16) &&
         p.y_ld % 8 == 0 && !(((uintptr_t)p.u | (uintptr_t)p.y | (uintptr_t)p.w) & 15);
}

}  // namespace

#define LMX_RG_KS(F)                                                                  \
  switch (bp / 32) {                                                                  \
    case 1: F(1); break;                                                              \
    case 2: F(2); break;                                                              \
    case 4: F(4); break;                                                              \
    case 8: F(8); break;                                                              \
    default: F(16);                                                                   \
  }

int rglru_chunks(const void* u, const void* y, long y_ld, const float* y_b, const float* g_b,
                 const float* log_a, void* out, float* state, const int* cu_q, const int* ctx,
                 const int* slots, int C, int bp, const void* w, int seq0, const int* segs,
                 int nsegs, const int* first, float* ws, hipStream_t stream) {
  if (nsegs <= 0) return 0;
  const RglruArgs p{u, y, y_ld, y_b, g_b, log_a, out, state, cu_q, ctx, slots, C, bp,
                    (const bf16_t*)w};
  if (!rglru_ok(p, true)) return -1;
  const dim3 grid(nsegs, (C + CT - 1) / CT);
#define LMX_RG_P(KS, PASS)                                                            \
  {                                                                                   \
    constexpr int smem = 2 * (TC * (KS == 1 ? 64 : KS * 32) + TC * CT) * 2;           \
    static bool attr = false;                                                         \
    if (smem > 65536 && !attr) {                                                      \
      (void)hipFuncSetAttribute((const void*)rglru_chunk_kernel<KS, PASS>,            \
                                hipFuncAttributeMaxDynamicSharedMemorySize, smem);    \
      attr = true;                                                                    \
    }                                                                                 \
    rglru_chunk_kernel<KS, PASS><<<grid, dim3(256), smem, stream>>>(p, seq0, segs,    \
                                                                    nsegs, first, ws); \
  }
#define LMX_RG(KS)                                                                    \
  if (ws) { LMX_RG_P(KS, 1) LMX_RG_P(KS, 2) } else { LMX_RG_P(KS, 0) }
  LMX_RG_KS(LMX_RG)
#undef LMX_RG
#undef LMX_RG_P
  return (int)hipGetLastError();
}

int rglru_rows(const void* u, const void* y, long y_ld, const float* y_b, const float* g_b,
               const float* log_a, void* out, float* state, const int* cu_q, const int* ctx,
               const int* slots, int C, int bp, const void* w, int rows, hipStream_t stream) {
  if (rows <= 0) return 0;
  const RglruArgs p{u, y, y_ld, y_b, g_b, log_a, out, state, cu_q, ctx, slots, C, bp,
                    (const bf16_t*)w};
  if (!rglru_ok(p, true)) return -1;
  const dim3 grid((C + CT - 1) / CT, (rows + 15) / 16);
#define LMX_RG(KS) rglru_rows_kernel<KS><<<grid, dim3(256), 0, stream>>>(p, rows)
  LMX_RG_KS(LMX_RG)
#undef LMX_RG
  return (int)hipGetLastError();
}

int rglru_scan(const void* u, const void* y, long y_ld, const float* y_b, const float* g_b,
               const float* log_a, void* out, float* state, const int* cu_q, const int* ctx,
               const int* slots, int C, int bp, const float* z, int S, int is_bf16,
               hipStream_t stream) {
  if (S <= 0) return 0;
  const RglruArgs p{u, y, y_ld, y_b, g_b, log_a, out, state, cu_q, ctx, slots, C, bp, nullptr};
  if (!rglru_ok(p, false)) return -1;
  const dim3 grid(S, (C + 63) / 64);
  if (is_bf16) rglru_scan_kernel<bf16_t><<<grid, dim3(64), 0, stream>>>(p, z);
  else rglru_scan_kernel<float><<<grid, dim3(64), 0, stream>>>(p, z);
  return (int)hipGetLastError();
}

}  // namespace lmx
