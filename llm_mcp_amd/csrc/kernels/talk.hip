// K22: paged attention with talking heads: the heads' scores are mixed before the
// softmax, score_h <- sum_g mix[h][g] score_g, so a row's heads run together; a
// sink per head adds exp(sink_h) to the softmax's denominator; a row sees the
// positions up to its own of its chunk (counted from position 0; 0: all of
// them); the output is multiplied by out_scale sigmoid(gate).  Query rows carry
// their scale.
//
// bf16 rows on MFMA, fp32 everywhere else: raw scores enter the mixing product,
// and softmax weights the product with V, as a bf16 pair (high part + remainder,
// 2^-17); the mix is bf16 as stored.
//   talk_prefill  8 query rows x all heads per workgroup, a 32-key page at a
//                 time: wave w scores its heads (columns = queries), the raw
//                 scores go through LDS to the wave that mixes and softmaxes one
//                 query's heads (columns = heads), the weights go back through
//                 LDS to the heads' waves for the product with V.
//   talk_decode   one row per workgroup, wave w = key heads w, w + W, ..: raw
//                 scores of a page through LDS, then every wave mixes its own
//                 heads and keeps their softmax and output, as K4 does.  Long
//                 chunks are split over workgroups, talk_reduce joins them.
//   talk_any      any geometry, fp32: one wave per row and head, scoring the
//                 mixed query (sum_g mix[h][g] q_g per key head) against all key
//                 heads.
#include <algorithm>

#include "attention.h"

namespace lmx {
namespace {

struct TalkArgs {
  const void* q;             // [rows][Hq * D]
  const void *kc, *vc;
  const void* mix;           // [Hq][Hq]
  const float* sink;         // [Hq]
  const int* bt;
  int bt_stride;
  const void* gate;
  long gate_ld;
  void* out;
  long out_ld;
  float out_scale;
  int Hq, Hkv, chunk;
};

// first position that a row at position p sees
__device__ __forceinline__ int chunk_first(int chunk, int p) { return chunk ? p / chunk * chunk : 0; }

// LDS images of [row groups of 16][32 rows][8 pieces of 16 B]: bytes of piece p
// (0..3 high parts, 4..7 remainders of 32 values) of row r in group q.  16 rows of
// a group, and 16 groups of a row, fall on 16 different pieces of the banks.
__device__ __forceinline__ int pair_off(int q, int r, int p) {
  return (q * 16 + (r >> 1)) * 256 + 16 * ((((r & 1) << 3) | p) ^ (q & 15) ^ ((r >> 1) & 7));
}
constexpr int PAIR_GROUP = 16 * 256;           // bytes of one group

// mixing operand: lane (column h, k = 8 g + j) = mix[h][k]
__device__ __forceinline__ bf16x8_t mix_frag(const bf16_t* mix, int Hq, int h, bool on, int g) {
  bf16x8_t f = {0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
  for (int j = 0; j < 8; ++j)
    if (on && 8 * g + j < Hq) f[j] = (short)mix[(long)h * Hq + 8 * g + j];
  return f;
}

__device__ __forceinline__ void split1(float x, uint16_t& hi, uint16_t& lo) {
  hi = f2bf(x);
  lo = f2bf(x - bf2f(hi));
}

// two values to packed bf16, one instruction
__device__ __forceinline__ uint32_t cvt_pk(float a, float b) {
  uint32_t r;
  asm("v_cvt_pk_bf16_f32 %0, %1, %2" : "=v"(r) : "v"(a), "v"(b));
  return r;
}
__device__ __forceinline__ void split2(float a, float b, uint32_t& hi, uint32_t& lo) {
  hi = cvt_pk(a, b);
  lo = cvt_pk(a - __uint_as_float(hi << 16), b - __uint_as_float(hi & 0xffff0000u));
}

// four outputs of a row's head times the gate
__device__ __forceinline__ void store_gated(const TalkArgs& a, long row, long col, const f32x4_t& o) {
  const bf16x4_t gv = *reinterpret_cast<const bf16x4_t*>((const bf16_t*)a.gate + row * a.gate_ld + col);
  bf16x4_t w;
#pragma unroll
  for (int r = 0; r < 4; ++r)
    w[r] = (short)f2bf(o[r] * a.out_scale *
                       __builtin_amdgcn_rcpf(1.f + fast_exp2(-LOG2E * bf2f((uint16_t)gv[r]))));
  *reinterpret_cast<bf16x4_t*>((bf16_t*)a.out + row * a.out_ld + col) = w;
}

// --------------------------------------------------------------- prefill ----
constexpr int TQ = 8;        // query rows per workgroup
constexpr int TW = 8;        // waves

// HPW: heads per wave (Hq <= 8 HPW), from h0 = HPW wave on.  A column group is 8
// queries (c % 8) x two heads (c / 8): group i holds head h0 + 2 (c / 8) + i of 4,
// h0 + c / 8 of 2, h0 of 1 (its other half idle).  Between two barriers a wave
// scores the next page, mixes this one and weighs the one before, through two
// images each.  SHARED: a wave's heads have one key head, whose pages are loaded
// ahead: K once a page's scores are made, V once its product is.  grid (tiles),
// block 512.
template <int HD, int HPW, bool SHARED>
__global__ void __launch_bounds__(64 * TW, 2) talk_prefill_kernel(
    TalkArgs a, const int* __restrict__ cu_q, const int* __restrict__ ctx_lens,
    const int* __restrict__ tiles) {
  extern __shared__ __attribute__((aligned(16))) char talk_sm[];
  constexpr int KS = HD / 32, NT = HD / 16, HT = HPW > 1 ? HPW / 2 : 1, NG = HPW == 4 ? 2 : 1;
  constexpr int IMG = TQ * PAIR_GROUP;
  char* const sS = talk_sm;                              // 2 x raw scores: group = query, row = key
  char* const sP = talk_sm + 2 * IMG;                    // 2 x weights: group = query, row = head
  float* const sAl = reinterpret_cast<float*>(sP + 2 * IMG);    // 2 x [32 heads][8]
  const int tile = blockIdx.x;
  const int seq = tiles[2 * tile], q0 = tiles[2 * tile + 1];
  const int lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4, cq = c & 7, cs = c >> 3;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int qbeg = cu_q[seq], qlen = cu_q[seq + 1] - qbeg, ctx = ctx_lens[seq];
  const int p0 = ctx - qlen + q0, p1 = ctx - qlen + min(q0 + TQ, qlen) - 1;   // positions
  const int pg0 = chunk_first(a.chunk, p0) / BS, pg1 = p1 / BS;
  const int* bt = a.bt + (long)seq * a.bt_stride;
  const int Hq = a.Hq, Hkv = a.Hkv, G = Hq / Hkv, h0 = wave * HPW;
  const bf16_t* kc = (const bf16_t*)a.kc;
  const bf16_t* vc = (const bf16_t*)a.vc;
  auto head = [&](int i, int s) { return h0 + (HPW == 4 ? 2 * s + i : HPW == 2 ? s : 0); };
  auto mine = [&](int i) { return head(i, cs) < Hq && (HPW > 1 || cs == 0); };   // this lane's column

  if constexpr (HPW < 4) {                               // heads that do not exist
    for (int i = threadIdx.x; i < 2 * IMG / 16; i += 64 * TW)
      reinterpret_cast<f32x4_t*>(sS)[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  }

  bf16x8_t qf[NG][KS];
#pragma unroll
  for (int i = 0; i < NG; ++i) {
    const bool on = mine(i) && q0 + cq < qlen;
    const bf16_t* qr = (const bf16_t*)a.q +
                       ((long)(qbeg + (on ? q0 + cq : 0)) * Hq + (on ? head(i, cs) : 0)) * HD;
#pragma unroll
    for (int s = 0; s < KS; ++s)
      qf[i][s] = on ? load_frag16B(qr + 32 * s + 8 * g) : bf16x8_t{0, 0, 0, 0, 0, 0, 0, 0};
  }
  // mixing: query `wave`, heads as columns
  bf16x8_t mf[HT];
  float m[HT], l[HT];
#pragma unroll
  for (int t = 0; t < HT; ++t) {
    const int h = 16 * t + c;
    mf[t] = mix_frag((const bf16_t*)a.mix, Hq, h, h < Hq, g);
    m[t] = h < Hq ? a.sink[h] * LOG2E : 0.f;             // the sink opens the sum
    l[t] = 1.f;
  }
  const int lim = q0 + wave < qlen ? ctx - qlen + q0 + wave : -1;
  const int lo = chunk_first(a.chunk, max(lim, 0));
  f32x4_t acc[NG][NT];
#pragma unroll
  for (int i = 0; i < NG; ++i)
#pragma unroll
    for (int n = 0; n < NT; ++n) acc[i][n] = f32x4_t{0.f, 0.f, 0.f, 0.f};

  bf16x8_t ka[KS], kb[KS], vf[NT];
  const int kvw = min(h0, Hq - 1) / G;                   // SHARED: the wave's key head
  auto load_k = [&](long blk, int kv) {
    const bf16_t* kp = kc + (blk * Hkv + kv) * (BS * HD);
#pragma unroll
    for (int t = 0; t < KS; ++t) {
      ka[t] = load_frag16B(kp + c * HD + 32 * t + 8 * g);
      kb[t] = load_frag16B(kp + (16 + c) * HD + 32 * t + 8 * g);
    }
  };
  auto load_v = [&](long blk, int kv) {
    const bf16_t* vp = vc + (blk * Hkv + kv) * (BS * HD);
#pragma unroll
    for (int n = 0; n < NT; ++n)
      vf[n] = load_frag_2x8B(vp + vq_off(16 * n + c, 8 * g, HD), vp + vq_off(16 * n + c, 8 * g + 4, HD));
  };
  // raw scores of the wave's heads: rows = keys, columns = (head, query)
  auto score = [&](int pg, char* img, int ahead) {       // ahead: block of the page to load
    f32x4_t s[NG][2];
#pragma unroll
    for (int i = 0; i < NG; ++i) {
      s[i][0] = s[i][1] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      if constexpr (SHARED) {
#pragma unroll
        for (int t = 0; t < KS; ++t) {
          s[i][0] = mfma16(ka[t], qf[i][t], s[i][0]);
          s[i][1] = mfma16(kb[t], qf[i][t], s[i][1]);
        }
      } else {
        const long blk = bt[pg];
#pragma unroll
        for (int half = 0; half < 2; ++half) {
          load_k(blk, min(head(i, half), Hq - 1) / G);
          f32x4_t x = {0.f, 0.f, 0.f, 0.f}, y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int t = 0; t < KS; ++t) {
            x = mfma16(ka[t], qf[i][t], x);
            y = mfma16(kb[t], qf[i][t], y);
          }
          s[i][0] = cs == half ? x : s[i][0];
          s[i][1] = cs == half ? y : s[i][1];
        }
      }
    }
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = 16 * b + 4 * g + r, h = head(0, cs);
        char* ph = img + pair_off(cq, key, h >> 3) + 2 * (h & 7);
        char* pl = img + pair_off(cq, key, 4 + (h >> 3)) + 2 * (h & 7);
        if constexpr (NG == 2) {
          uint32_t hi, lw;
          split2(s[0][b][r], s[NG - 1][b][r], hi, lw);
          *reinterpret_cast<uint32_t*>(ph) = hi;
          *reinterpret_cast<uint32_t*>(pl) = lw;
        } else {
          uint16_t hi, lw;
          split1(s[0][b][r], hi, lw);
          if (HPW > 1 || cs == 0) {
            *reinterpret_cast<uint16_t*>(ph) = hi;
            *reinterpret_cast<uint16_t*>(pl) = lw;
          }
        }
      }
    if (SHARED) load_k(ahead, kvw);
  };
  // a query: mix (rows = keys, columns = heads), softmax
  auto mix = [&](int pg, const char* img, char* pimg, float* al_img) {
    f32x4_t x[HT][2];
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      const bf16x8_t sh = *reinterpret_cast<const bf16x8_t*>(img + pair_off(wave, 16 * b + c, g));
      const bf16x8_t sl = *reinterpret_cast<const bf16x8_t*>(img + pair_off(wave, 16 * b + c, 4 + g));
#pragma unroll
      for (int t = 0; t < HT; ++t) {
        x[t][b] = mfma16(sh, mf[t], f32x4_t{0.f, 0.f, 0.f, 0.f});
        x[t][b] = mfma16(sl, mf[t], x[t][b]);
      }
    }
    // a page of which every key is seen needs no mask
    if (pg * BS + BS - 1 > lim || pg * BS < lo) {
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int key = pg * BS + 16 * b + 4 * g + r;
#pragma unroll
          for (int t = 0; t < HT; ++t)
            if (key > lim || key < lo) x[t][b][r] = -INFINITY;
        }
    }
#pragma unroll
    for (int t = 0; t < HT; ++t) {
      const f32x4_t &u = x[t][0], &v = x[t][1];
      const float mx = max3f(max3f(u[0], u[1], u[2]), max3f(u[3], v[0], v[1]), max2f(v[2], v[3]));
      const float mn = max2f(m[t], col4_max(mx) * LOG2E);
      const float al = fast_exp2(m[t] - mn);
      m[t] = mn;
      float sum = 0.f;
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        float w[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          w[r] = fast_exp2(x[t][b][r] * LOG2E - mn);
          sum += w[r];
        }
        uint32_t h01, l01, h23, l23;
        split2(w[0], w[1], h01, l01);
        split2(w[2], w[3], h23, l23);
        const int h = 16 * t + c, piece = 2 * b + (g >> 1), sub = 8 * (g & 1);
        *reinterpret_cast<uint2*>(pimg + pair_off(wave, h, piece) + sub) = make_uint2(h01, h23);
        *reinterpret_cast<uint2*>(pimg + pair_off(wave, h, 4 + piece) + sub) = make_uint2(l01, l23);
      }
      l[t] = l[t] * al + col4_sum(sum);
      if (g == 0) al_img[(16 * t + c) * TQ + wave] = al;
    }
  };
  // weights times V: rows = channels, columns = (head, query)
  auto weigh = [&](int pg, const char* pimg, const float* al_img, int ahead) {
#pragma unroll
    for (int i = 0; i < NG; ++i) {
      const int h = head(i, cs);                       // beyond Hq: a row of the image all the same
      const bf16x8_t ph = *reinterpret_cast<const bf16x8_t*>(pimg + pair_off(cq, h, g));
      const bf16x8_t pl = *reinterpret_cast<const bf16x8_t*>(pimg + pair_off(cq, h, 4 + g));
      const float al = al_img[h * TQ + cq];
#pragma unroll
      for (int n = 0; n < NT; ++n) acc[i][n] *= al;
      if constexpr (SHARED) {
#pragma unroll
        for (int n = 0; n < NT; ++n) {
          acc[i][n] = mfma16(vf[n], ph, acc[i][n]);
          acc[i][n] = mfma16(vf[n], pl, acc[i][n]);
        }
      } else {
        const bf16x8_t zero = {0, 0, 0, 0, 0, 0, 0, 0};
        const long blk = bt[pg];
#pragma unroll
        for (int half = 0; half < 2; ++half) {
          load_v(blk, min(head(i, half), Hq - 1) / G);
#pragma unroll
          for (int n = 0; n < NT; ++n) {
            acc[i][n] = mfma16(vf[n], cs == half ? ph : zero, acc[i][n]);
            acc[i][n] = mfma16(vf[n], cs == half ? pl : zero, acc[i][n]);
          }
        }
      }
    }
    if (SHARED) load_v(ahead, kvw);
  };
  // block ids: lane i holds page base + i
  int base = pg0, ids = bt[min(pg0 + lane, pg1)];
  asm volatile("" : "+v"(ids));                          // landed before the loop's loads are counted
  auto page = [&](int pg) { return __builtin_amdgcn_readlane(ids, min(pg, pg1) - base); };
  if (SHARED) load_k(page(pg0), kvw);
  lds_barrier();                                         // the zeros are in place
  score(pg0, sS, page(pg0 + 1));
  lds_barrier();
  score(min(pg0 + 1, pg1), sS + IMG, page(pg0 + 2));
  // in the order of the loop's loads, K before V: the waits are counted
  __builtin_amdgcn_sched_barrier(0);
  if (SHARED) load_v(page(pg0), kvw);
  mix(pg0, sS, sP, sAl);
  lds_barrier();
  int cur = 1;                                           // image of this page
  for (int pg = pg0 + 1; pg <= pg1; ++pg, cur ^= 1) {
    if (pg - base >= 32) {
      base = pg;
      ids = bt[min(pg + lane, pg1)];
      asm volatile("" : "+v"(ids));
    }
    score(min(pg + 1, pg1), sS + (cur ^ 1) * IMG, page(pg + 2));
    mix(pg, sS + cur * IMG, sP + cur * IMG, sAl + cur * 32 * TQ);
    weigh(pg - 1, sP + (cur ^ 1) * IMG, sAl + (cur ^ 1) * 32 * TQ, page(pg));
    lds_barrier();
  }
  weigh(pg1, sP + (cur ^ 1) * IMG, sAl + (cur ^ 1) * 32 * TQ, page(pg1));
  // the weights' sums go to the heads' waves
  lds_barrier();
#pragma unroll
  for (int t = 0; t < HT; ++t)
    if (g == 0) sAl[(16 * t + c) * TQ + wave] = 1.f / l[t];
  lds_barrier();
  if (q0 + cq < qlen) {
    const long row = qbeg + q0 + cq;
#pragma unroll
    for (int i = 0; i < NG; ++i) {
      if (!mine(i)) continue;
      const int h = head(i, cs);
      const float inv = sAl[h * TQ + cq];
#pragma unroll
      for (int n = 0; n < NT; ++n)
        store_gated(a, row, (long)h * HD + 16 * n + 4 * g, acc[i][n] * inv);
    }
  }
}

// ---------------------------------------------------------------- decode ----
// keys per partition: whole pages, at most max_parts partitions
__device__ __forceinline__ int decode_part(int n, int part_tokens, int max_parts) {
  return max(part_tokens, ((n + max_parts - 1) / max_parts + BS - 1) / BS * BS);
}

// grid (max_parts, rows), block 64 * min(8, Hkv); KPW: key heads per wave
template <int HD, int KPW>
__global__ void __launch_bounds__(512) talk_decode_kernel(TalkArgs a, const int* __restrict__ ctx_lens,
                                                          float* __restrict__ part_o,
                                                          float* __restrict__ part_ml,
                                                          int part_tokens, int max_parts) {
  __shared__ __attribute__((aligned(16))) char sS[2][PAIR_GROUP];
  constexpr int KS = HD / 32, NT = HD / 16;
  const int b = blockIdx.y, p = blockIdx.x;
  const int ctx = ctx_lens[b], lo = chunk_first(a.chunk, ctx - 1), base = lo / BS * BS;
  const int part = decode_part(ctx - base, part_tokens, max_parts);
  const int nparts = (ctx - base + part - 1) / part;
  if (p >= nparts) return;
  const int lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), W = blockDim.x >> 6;
  const int Hq = a.Hq, Hkv = a.Hkv, G = Hq / Hkv;
  const bf16_t* kc = (const bf16_t*)a.kc;
  const bf16_t* vc = (const bf16_t*)a.vc;
  const int* bt = a.bt + (long)b * a.bt_stride;
  const int t0 = base + p * part, t1 = min(t0 + part, ctx);
  const int pg0 = t0 / BS, pg1 = (t1 + BS - 1) / BS;

  for (int i = threadIdx.x; i < 2 * PAIR_GROUP / 16; i += blockDim.x)  // heads that do not exist
    reinterpret_cast<f32x4_t*>(sS)[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  bf16x8_t qf[KPW][KS], mf[KPW];
  float m[KPW], l[KPW];
  f32x4_t acc[KPW][NT];
#pragma unroll
  for (int i = 0; i < KPW; ++i) {
    const int kv = wave + i * W, h = kv * G + c;
    const bool on = kv < Hkv && c < G;
    const bf16_t* qr = (const bf16_t*)a.q + ((long)b * Hq + (on ? h : 0)) * HD;
#pragma unroll
    for (int s = 0; s < KS; ++s)
      qf[i][s] = on ? load_frag16B(qr + 32 * s + 8 * g) : bf16x8_t{0, 0, 0, 0, 0, 0, 0, 0};
    mf[i] = mix_frag((const bf16_t*)a.mix, Hq, h, on, g);
    m[i] = -INFINITY;
    l[i] = 0.f;
#pragma unroll
    for (int n = 0; n < NT; ++n) acc[i][n] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  }
  bf16x8_t ka[KS], kb[KS];             // one key head per wave: a page ahead
  auto load_k = [&](long blk, int kv) {
    const bf16_t* kp = kc + (blk * Hkv + min(kv, Hkv - 1)) * (BS * HD);
#pragma unroll
    for (int t = 0; t < KS; ++t) {
      ka[t] = load_frag16B(kp + c * HD + 32 * t + 8 * g);
      kb[t] = load_frag16B(kp + (16 + c) * HD + 32 * t + 8 * g);
    }
  };
  if (KPW == 1) load_k(bt[pg0], wave);
  lds_barrier();
  for (int pg = pg0; pg < pg1; ++pg) {
    char* const img = sS[(pg - pg0) & 1];
    const long blk = bt[pg];
    bf16x8_t vf[KPW == 1 ? NT : 1];
    if constexpr (KPW == 1) {
      const bf16_t* vp = vc + (blk * Hkv + wave) * (BS * HD);
#pragma unroll
      for (int n = 0; n < NT; ++n)
        vf[n] = load_frag_2x8B(vp + vq_off(16 * n + c, 4 * g, HD), vp + vq_off(16 * n + c, 16 + 4 * g, HD));
    }
    // raw scores: rows = the key head's query heads, columns = keys
#pragma unroll
    for (int i = 0; i < KPW; ++i) {
      if (KPW > 1) __builtin_amdgcn_sched_barrier(0);    // one key head's operands at a time
      const int kv = wave + i * W;
      f32x4_t s[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
      if (KPW > 1) load_k(blk, kv);
#pragma unroll
      for (int t = 0; t < KS; ++t) {
        s[0] = mfma16(qf[i][t], ka[t], s[0]);
        s[1] = mfma16(qf[i][t], kb[t], s[1]);
      }
      if (kv < Hkv) {
#pragma unroll
        for (int x = 0; x < 2; ++x)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            if (4 * g + r >= G) continue;
            const int h = kv * G + 4 * g + r;
            uint16_t hi, lw;
            split1(s[x][r], hi, lw);
            *reinterpret_cast<uint16_t*>(img + pair_off(0, 16 * x + c, h >> 3) + 2 * (h & 7)) = hi;
            *reinterpret_cast<uint16_t*>(img + pair_off(0, 16 * x + c, 4 + (h >> 3)) + 2 * (h & 7)) = lw;
          }
      }
    }
    if (KPW == 1 && pg + 1 < pg1) load_k(bt[pg + 1], wave);
    lds_barrier();
    bf16x8_t sh[2], sl[2];
#pragma unroll
    for (int x = 0; x < 2; ++x) {
      sh[x] = *reinterpret_cast<const bf16x8_t*>(img + pair_off(0, 16 * x + c, g));
      sl[x] = *reinterpret_cast<const bf16x8_t*>(img + pair_off(0, 16 * x + c, 4 + g));
    }
#pragma unroll
    for (int i = 0; i < KPW; ++i) {
      if (KPW > 1) __builtin_amdgcn_sched_barrier(0);
      const int kv = min(wave + i * W, Hkv - 1);
      float x[8], mx = -INFINITY;
#pragma unroll
      for (int y = 0; y < 2; ++y) {
        f32x4_t s = mfma16(sh[y], mf[i], f32x4_t{0.f, 0.f, 0.f, 0.f});
        s = mfma16(sl[y], mf[i], s);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int key = pg * BS + 16 * y + 4 * g + r;
          x[4 * y + r] = key < t1 && key >= lo ? s[r] * LOG2E : -INFINITY;
          mx = fmaxf(mx, x[4 * y + r]);
        }
      }
      const float mn = fmaxf(m[i], col4_max(mx)), mu = mn == -INFINITY ? 0.f : mn;
      const float al = fast_exp2(m[i] - mu);
      float w[8], sum = 0.f;
#pragma unroll
      for (int j = 0; j < 8; ++j) { w[j] = fast_exp2(x[j] - mu); sum += w[j]; }
      m[i] = mn;
      l[i] = l[i] * al + col4_sum(sum);
      bf16x8_t ph, pl;
      split_weights(w, ph, pl);
      const bf16_t* vp = vc + (blk * Hkv + kv) * (BS * HD);
#pragma unroll
      for (int n = 0; n < NT; ++n) {
        bf16x8_t v;
        if constexpr (KPW == 1) v = vf[n];
        else v = load_frag_2x8B(vp + vq_off(16 * n + c, 4 * g, HD), vp + vq_off(16 * n + c, 16 + 4 * g, HD));
        acc[i][n] *= al;
        acc[i][n] = mfma16(v, ph, acc[i][n]);
        acc[i][n] = mfma16(v, pl, acc[i][n]);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < KPW; ++i) {
    const int kv = wave + i * W, h = kv * G + c;
    if (kv >= Hkv || c >= G) continue;
    if (nparts == 1) {
      const float sk = a.sink[h] * LOG2E, M = fmaxf(m[i], sk);
      const float f = fast_exp2(m[i] - M), inv = f / (l[i] * f + fast_exp2(sk - M));
#pragma unroll
      for (int n = 0; n < NT; ++n)
        store_gated(a, b, (long)h * HD + 16 * n + 4 * g, acc[i][n] * inv);
    } else {
      const long idx = ((long)b * Hq + h) * max_parts + p;
#pragma unroll
      for (int n = 0; n < NT; ++n)
        *reinterpret_cast<f32x4_t*>(part_o + idx * HD + 16 * n + 4 * g) = acc[i][n];
      if (g == 0) { part_ml[idx * 2] = m[i]; part_ml[idx * 2 + 1] = l[i]; }
    }
  }
}

// grid (Hq, rows), block HD / 4: joins the partitions of a row and the sink
template <int HD>
__global__ void __launch_bounds__(64) talk_reduce_kernel(TalkArgs a, const int* __restrict__ ctx_lens,
                                                         const float* __restrict__ part_o,
                                                         const float* __restrict__ part_ml,
                                                         int part_tokens, int max_parts) {
  const int h = blockIdx.x, b = blockIdx.y, d = 4 * threadIdx.x;
  const int ctx = ctx_lens[b], n = ctx - chunk_first(a.chunk, ctx - 1) / BS * BS;
  const int part = decode_part(n, part_tokens, max_parts);
  const int nparts = (n + part - 1) / part;
  if (nparts <= 1) return;
  const long at = ((long)b * a.Hq + h) * max_parts;
  const float sk = a.sink[h] * LOG2E;
  float M = sk;
  for (int p = 0; p < nparts; ++p) M = fmaxf(M, part_ml[(at + p) * 2]);
  float L = fast_exp2(sk - M);
  f32x4_t O = {0.f, 0.f, 0.f, 0.f};
  for (int p = 0; p < nparts; ++p) {
    const float f = fast_exp2(part_ml[(at + p) * 2] - M);
    L += part_ml[(at + p) * 2 + 1] * f;
    O += *reinterpret_cast<const f32x4_t*>(part_o + (at + p) * HD + d) * f;
  }
  store_gated(a, b, (long)h * HD + d, O * (1.f / L));
}

// ------------------------------------------------------ any head geometry ----
// One wave per (row, query head): the mixed query in LDS, a lane per key of a
// 64-key block, then every 64th output channel per lane.
// grid (rows, ceil(Hq / waves)), LDS: waves x Hkv x D floats
template <typename T, int ND>
__global__ void __launch_bounds__(256) talk_any_kernel(TalkArgs a, const int* __restrict__ cu_q, int S,
                                                       const int* __restrict__ positions) {
  extern __shared__ float any_sm[];
  constexpr int D = ND * 64;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int row = blockIdx.x, h = blockIdx.y * (blockDim.x >> 6) + wave;
  const int Hq = a.Hq, Hkv = a.Hkv, G = Hq / Hkv;
  const bool on = h < Hq;
  float* sq = any_sm + (long)wave * Hkv * D;
  if (on)
    for (int x = lane; x < Hkv * D; x += 64) {
      const int kv = x / D, d = x - kv * D;
      const T* qr = (const T*)a.q + ((long)row * Hq + kv * G) * D + d;
      const T* mr = (const T*)a.mix + (long)h * Hq + kv * G;
      float s = 0.f;
      for (int j = 0; j < G; ++j) s += ld1(mr + j) * ld1(qr + (long)j * D);
      sq[x] = s;
    }
  __syncthreads();
  if (!on) return;
  int lo = 0, hi = S - 1;                     // the sequence of this row
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (cu_q[mid] <= row) lo = mid; else hi = mid - 1;
  }
  const int* tab = a.bt + (long)lo * a.bt_stride;
  const int n = positions[row] + 1;
  const long kvh = h / G;
  float m = a.sink[h], l = 1.f, acc[ND];
#pragma unroll
  for (int i = 0; i < ND; ++i) acc[i] = 0.f;
  for (int k0 = chunk_first(a.chunk, n - 1); k0 < n; k0 += 64) {
    const int key = k0 + lane;
    float s = -INFINITY;
    if (key < n) {
      float t = 0.f;
      for (int kv = 0; kv < Hkv; ++kv) {
        const T* kp = (const T*)a.kc + (((long)tab[key / BS] * Hkv + kv) * BS + key % BS) * D;
        for (int d = 0; d < D; d += 8) {
          float x[8];
          ldv<8>(x, kp + d);
#pragma unroll
          for (int e = 0; e < 8; ++e) t += x[e] * sq[kv * D + d + e];
        }
      }
      s = t;
    }
    const float mn = fmaxf(m, wave_max(s));
    const float al = expf(m - mn), p = expf(s - mn);   // exp(-inf) = 0
    l = l * al + wave_sum(p);
    m = mn;
#pragma unroll
    for (int i = 0; i < ND; ++i) acc[i] *= al;
    const int cnt = min(64, n - k0);
    for (int j = 0; j < cnt; ++j) {
      const float pj = __shfl(p, j, 64);
      const int kj = k0 + j, off = kj % BS;
      const T* vp = (const T*)a.vc + ((long)tab[kj / BS] * Hkv + kvh) * BS * D;
#pragma unroll
      for (int i = 0; i < ND; ++i) acc[i] += pj * ld1(vp + vq_off(i * 64 + lane, off, D));
    }
  }
  const float inv = a.out_scale / l;
#pragma unroll
  for (int i = 0; i < ND; ++i) {
    const long col = (long)h * D + i * 64 + lane;
    const float gt = sigmoid_t<T>(ld1((const T*)a.gate + row * a.gate_ld + col));
    st1((T*)a.out + row * a.out_ld + col, acc[i] * inv * gt);
  }
}

bool talk_ok(const TalkArgs& a, int D) {
  return a.q && a.kc && a.vc && a.mix && a.sink && a.gate && a.out && a.Hkv > 0 && a.Hq > 0 &&
         a.Hq % a.Hkv == 0 && a.chunk >= 0 && (D == 64 || D == 128 || D == 256 || D == 512);
}
// the MFMA forms: one mixing step of 32 heads, 16-B rows
bool talk_mfma_ok(const TalkArgs& a, int D) {
  return talk_ok(a, D) && D <= 128 && a.Hq <= 32 && a.Hq / a.Hkv <= 16 && a.gate_ld % 8 == 0 &&
         a.out_ld % 8 == 0 && !(((uintptr_t)a.q | (uintptr_t)a.gate | (uintptr_t)a.out) & 15);
}

template <int HD, int HPW, bool SHARED>
int launch_prefill_as(const TalkArgs& a, const int* cu_q, const int* ctx, const int* tiles, int n,
                      hipStream_t stream) {
  constexpr int smem = 4 * TQ * PAIR_GROUP + 2 * 32 * TQ * 4;
  static bool attr = false;
  if (!attr) {
    const hipError_t e = hipFuncSetAttribute((const void*)talk_prefill_kernel<HD, HPW, SHARED>,
                                             hipFuncAttributeMaxDynamicSharedMemorySize, smem);
    if (e != hipSuccess) return (int)e;
    attr = true;
  }
  talk_prefill_kernel<HD, HPW, SHARED><<<dim3(n), dim3(64 * TW), smem, stream>>>(a, cu_q, ctx, tiles);
  return (int)hipGetLastError();
}

template <int HD, int HPW>
int launch_prefill(const TalkArgs& a, const int* cu_q, const int* ctx, const int* tiles, int n,
                   hipStream_t stream) {
  if constexpr (HPW > 1)
    if (a.Hq / a.Hkv % HPW) return launch_prefill_as<HD, HPW, false>(a, cu_q, ctx, tiles, n, stream);
  return launch_prefill_as<HD, HPW, true>(a, cu_q, ctx, tiles, n, stream);
}

}  // namespace

// cu_q, ctx, bt: of the sequences that tiles [n][2] (sequence, first query row) name
int talk_prefill(const void* q, const void* kc, const void* vc, const void* mix, const float* sink,
                 float out_scale, int Hq, int Hkv, int D, int chunk, const int* bt, int bt_stride,
                 const int* cu_q, const int* ctx, const int* tiles, int n, const void* gate,
                 long gate_ld, void* out, long out_ld, hipStream_t stream) {
  if (n <= 0) return 0;
  const TalkArgs a{q, kc, vc, mix, sink, bt, bt_stride, gate, gate_ld, out, out_ld, out_scale,
                   Hq, Hkv, chunk};
  if (!talk_mfma_ok(a, D)) return -1;
#define LMX_TP(HDV)                                                                   \
  return Hq <= 8    ? launch_prefill<HDV, 1>(a, cu_q, ctx, tiles, n, stream)          \
         : Hq <= 16 ? launch_prefill<HDV, 2>(a, cu_q, ctx, tiles, n, stream)          \
                    : launch_prefill<HDV, 4>(a, cu_q, ctx, tiles, n, stream);
  if (D == 64) { LMX_TP(64) } else { LMX_TP(128) }
#undef LMX_TP
}

int talk_decode(const void* q, const void* kc, const void* vc, const void* mix, const float* sink,
                float out_scale, int Hq, int Hkv, int D, int chunk, const int* bt, int bt_stride,
                const int* ctx, int rows, const void* gate, long gate_ld, void* out, long out_ld,
                float* part_o, float* part_ml, int part_tokens, int max_parts, hipStream_t stream) {
  if (rows <= 0) return 0;
  const TalkArgs a{q, kc, vc, mix, sink, bt, bt_stride, gate, gate_ld, out, out_ld, out_scale,
                   Hq, Hkv, chunk};
  if (!talk_mfma_ok(a, D) || Hkv > 32 || part_tokens < BS || part_tokens % BS || max_parts < 1 ||
      (max_parts > 1 && (!part_o || !part_ml)))
    return -1;
  const int waves = std::min(8, Hkv), kpw = (Hkv + waves - 1) / waves;
  const dim3 grid(max_parts, rows), block(64 * waves);
#define LMX_TD(HDV, K) \
  talk_decode_kernel<HDV, K><<<grid, block, 0, stream>>>(a, ctx, part_o, part_ml, part_tokens, max_parts)
#define LMX_TDH(HDV)                                                                          \
  if (kpw == 1) LMX_TD(HDV, 1); else if (kpw == 2) LMX_TD(HDV, 2); else LMX_TD(HDV, 4);       \
  if (max_parts > 1)                                                                          \
    talk_reduce_kernel<HDV><<<dim3(Hq, rows), dim3(HDV / 4), 0, stream>>>(a, ctx, part_o, part_ml, \
                                                                          part_tokens, max_parts);
  if (D == 64) { LMX_TDH(64) } else { LMX_TDH(128) }
#undef LMX_TDH
#undef LMX_TD
  return (int)hipGetLastError();
}

int talk_any(const void* q, const void* kc, const void* vc, const int* bt, int bt_stride,
             const int* cu_q, int S, const int* positions, int rows, const void* mix,
             const float* sink, void* out, long out_ld, const void* gate, long gate_ld,
             float out_scale, int Hq, int Hkv, int D, int chunk, int is_bf16, hipStream_t stream) {
  if (rows <= 0) return 0;
  const TalkArgs a{q, kc, vc, mix, sink, bt, bt_stride, gate, gate_ld, out, out_ld, out_scale,
                   Hq, Hkv, chunk};
  if (!talk_ok(a, D) || S < 1) return -1;
  const long per = (long)Hkv * D * 4;              // mixed query of one wave
  if (per > 160 * 1024) return -2;
  const int waves = 4 * per <= 65536 ? 4 : 1;
  const dim3 grid(rows, (Hq + waves - 1) / waves), block(64 * waves);
  const int smem = (int)(per * waves);
#define LMX_TA(T, ND)                                                                        \
  {                                                                                          \
    if (smem > 65536) {                                                                      \
      const hipError_t e = hipFuncSetAttribute((const void*)talk_any_kernel<T, ND>,          \
                                               hipFuncAttributeMaxDynamicSharedMemorySize, smem); \
      if (e != hipSuccess) return (int)e;                                                    \
    }                                                                                        \
    talk_any_kernel<T, ND><<<grid, block, smem, stream>>>(a, cu_q, S, positions);            \
  }
#define LMX_TAD(T) \
  if (D == 64) LMX_TA(T, 1) else if (D == 128) LMX_TA(T, 2) else if (D == 256) LMX_TA(T, 4) else LMX_TA(T, 8)
  if (is_bf16) { LMX_TAD(bf16_t) } else { LMX_TAD(float) }
#undef LMX_TAD
#undef LMX_TA
  return (int)hipGetLastError();
}

}  // namespace lmx
