// K16: short causal convolution over time, per channel, with the last
// (taps - 1) inputs of every sequence as state.
//
//   y_t[c] = sum_j w[j][c] u_{t - taps + 1 + j}[c]  (+ bias[c])
//
// with u the projection's rows plus, optionally, the projection's own bias
// (in_bias: the product itself then needs no bias pass).  u before a sequence's first token counts as zero; the inputs of tokens of
// earlier steps come from state[slots][taps - 1][C] (oldest first), which the
// step leaves holding the last taps - 1 inputs.  Two consumers share the walk:
//
//   short_conv      y (optionally SiLU) to a row tensor: the state-space
//                   mixer's x | B | C channels
//   conv_qkv_cache  the channels are padded q | k | v heads: q and k are
//                   divided by their root mean square over the head's true
//                   size (unit norm, no weight), q is multiplied by the
//                   position's temperature 1 + coef ln(floor((p+1)/every) + 1),
//                   q goes to a row tensor, k and v into their cache pages
//                   (rope_cache.hip layout) -- convolution, head norm,
//                   temperature and cache write in one pass over the
//                   projection rows
//
// A workgroup walks one tile of consecutive tokens of one sequence, V channels
// per thread, with the window of inputs in registers.  Only the tile at the
// start of a sequence's rows reads the state, and the same thread then writes
// it (a tile is at least taps - 1 tokens or the whole range), so no other
// workgroup races with the update.
#include "common.h"

namespace lmx {

struct ConvArgs {
  const void* u;        // T rows [.., C]
  long u_ld;
  const float* w;       // [taps][C]
  const float* in_bias; // [C] or null: added to u
  const float* bias;    // [C] or null: added to y
  void* state;          // T [slots][taps - 1][C]; null when taps == 1
  const int* tiles;     // [ntiles][2] (sequence, first row in it); null: one tile per sequence
  const int *cu_q, *ctx, *slots;
  int C, taps, tile;
};

// Walk of one tile: emit(row, y, last) per token.  TAPS > 0: window in registers;
// TAPS == 0: any tap count, inputs re-read (cache hits).
template <typename T, int V, int TAPS, typename Emit>
__device__ __forceinline__ void conv_walk(const ConvArgs& a, int seq, int start, int c0, Emit emit) {
  const int taps = TAPS ? TAPS : a.taps;
  const int row0 = a.cu_q[seq], n = a.cu_q[seq + 1] - row0;
  const bool fresh = a.ctx[seq] == n;
  const int end = min(start + a.tile, n);
  const T* u = (const T*)a.u + (long)row0 * a.u_ld + c0;
  T* st = a.state ? (T*)a.state + (long)a.slots[seq] * (taps - 1) * a.C + c0 : nullptr;
  // input at row r of this range (r < 0: an earlier token of the sequence)
  float ib[V];
#pragma unroll
  for (int e = 0; e < V; ++e) ib[e] = a.in_bias ? a.in_bias[c0 + e] : 0.f;
  auto input = [&](int r, float (&f)[V]) {
    if (r >= 0) {
      ldv<V>(f, u + (long)r * a.u_ld);
#pragma unroll
      for (int e = 0; e < V; ++e) f[e] += ib[e];
    } else if (!fresh) {
      ldv<V>(f, st + (long)(taps - 1 + r) * a.C);
    } else {
#pragma unroll
      for (int e = 0; e < V; ++e) f[e] = 0.f;
    }
  };
  float bias[V];
#pragma unroll
  for (int e = 0; e < V; ++e) bias[e] = a.bias ? a.bias[c0 + e] : 0.f;
  if constexpr (TAPS > 0) {
    float w[TAPS][V], win[TAPS][V], nxt[V];   // win[j]: input t - taps + 1 + j
#pragma unroll
    for (int j = 0; j < TAPS; ++j) ldv<V>(w[j], a.w + (long)j * a.C + c0);
#pragma unroll
    for (int j = 0; j < TAPS - 1; ++j) input(start - (TAPS - 1) + j, win[j]);
    input(start, nxt);
    for (int t = start; t < end; ++t) {
#pragma unroll
      for (int e = 0; e < V; ++e) win[TAPS - 1][e] = nxt[e];
      if (t + 1 < end) input(t + 1, nxt);     // in flight under this token's work
      float y[V];
#pragma unroll
      for (int e = 0; e < V; ++e) {
        float s = bias[e];
#pragma unroll
        for (int j = 0; j < TAPS; ++j) s += w[j][e] * win[j][e];
        y[e] = s;
      }
      emit(row0 + t, y, t + 1 == end);
#pragma unroll
      for (int j = 0; j + 1 < TAPS; ++j)
#pragma unroll
        for (int e = 0; e < V; ++e) win[j][e] = win[j + 1][e];
    }
  } else {
    for (int t = start; t < end; ++t) {
      float y[V];
#pragma unroll
      for (int e = 0; e < V; ++e) y[e] = bias[e];
      for (int j = 0; j < taps; ++j) {
        float w[V], x[V];
        ldv<V>(w, a.w + (long)j * a.C + c0);
        input(t - (taps - 1) + j, x);
#pragma unroll
        for (int e = 0; e < V; ++e) y[e] += w[e] * x[e];
      }
      emit(row0 + t, y, t + 1 == end);
    }
  }
  // state: inputs n - taps + 1 .. n - 1, written oldest first (entry s reads
  // an old entry only above s)
  if (start == 0 && taps > 1) {
    for (int s = 0; s < taps - 1; ++s) {
      float x[V];
      input(n - (taps - 1) + s, x);
      stv<V>(st + (long)s * a.C, x);
    }
  }
}

// grid (tiles, ceil(C / V / 256)), block 256
template <typename T, int V, int TAPS>
__global__ void __launch_bounds__(256) short_conv_kernel(ConvArgs a, void* out, long out_ld, int act) {
  const int seq = a.tiles ? a.tiles[2 * blockIdx.x] : blockIdx.x;
  const int start = a.tiles ? a.tiles[2 * blockIdx.x + 1] : 0;
  const int c0 = (blockIdx.y * 256 + threadIdx.x) * V;
  if (c0 >= a.C || a.slots[seq] < 0) return;
  conv_walk<T, V, TAPS>(a, seq, start, c0, [&](int row, float (&y)[V], bool) {
    if (act) {
#pragma unroll
      for (int e = 0; e < V; ++e) y[e] *= sigmoid_t<T>(y[e]);
    }
    stv<V>((T*)out + (long)row * out_ld + c0, y);
  });
}

struct QkvOut {
  void* q;              // T rows [.., Hq * D]
  long q_ld;
  void *kc, *vc;        // T pages [NB][Hkv][BS][D] / [NB][Hkv][BS/4][D][4]
  const int *positions, *slots;   // per row
  int Hq, Hkv, D, dk, BS;
  float eps, coef, every;
};

// grid (tiles, ceil(heads / (2048 / D))), block 256: D / 8 lanes per head
template <typename T, int TAPS>
__global__ void __launch_bounds__(256) conv_qkv_cache_kernel(ConvArgs a, QkvOut o) {
  const int seq = a.tiles ? a.tiles[2 * blockIdx.x] : blockIdx.x;
  const int start = a.tiles ? a.tiles[2 * blockIdx.x + 1] : 0;
  const int c0 = (blockIdx.y * 256 + threadIdx.x) * 8;
  if (c0 >= a.C || a.slots[seq] < 0) return;   // whole heads leave together
  const int head = c0 / o.D, d = c0 - head * o.D, lph = o.D >> 3;
  // bf16 v: the last 4 tokens of each channel, newest in the top 16 bits; a
  // key quad of the v page leaves as one 8-B store per channel
  unsigned long long vq[8];
  int vn = 0;                                  // tokens held since the walk began
  conv_walk<T, 8, TAPS>(a, seq, start, c0, [&](int row, float (&y)[8], bool last) {
    if (head < o.Hq + o.Hkv) {
      float ss = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) ss += y[e] * y[e];
      for (int m = 1; m < lph; m <<= 1) ss += __shfl_xor(ss, m, 64);
      float inv = rsqrtf(ss / (float)o.dk + o.eps);
      if (head < o.Hq) {
        const float p = (float)o.positions[row];
        inv *= 1.f + o.coef * logf(floorf((p + 1.f) / o.every) + 1.f);
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) y[e] *= inv;
    }
    if (head < o.Hq) {
      stv<8>((T*)o.q + (long)row * o.q_ld + c0, y);
      return;
    }
    const int slot = o.slots[row];
    if (slot < 0) return;
    const long blk = slot / o.BS;
    const int off = slot - (int)blk * o.BS;
    if (head < o.Hq + o.Hkv) {
      const long kvh = head - o.Hq;
      stv<8>((T*)o.kc + ((blk * o.Hkv + kvh) * o.BS + off) * o.D + d, y);
    } else {
      const long kvh = head - o.Hq - o.Hkv;
      T* vp = (T*)o.vc + (blk * o.Hkv + kvh) * o.BS * o.D + vq_off(d, off, o.D);
      if constexpr (sizeof(T) == 4) {
#pragma unroll
        for (int e = 0; e < 8; ++e) vp[4 * e] = y[e];
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e)
          vq[e] = (vn ? vq[e] >> 16 : 0ull) | (unsigned long long)f2bf(y[e]) << 48;
        ++vn;
        const int in_quad = (off & 3) + 1;     // tokens of this quad up to this one
        if (in_quad == 4 && vn >= 4) {
#pragma unroll
          for (int e = 0; e < 8; ++e) *reinterpret_cast<unsigned long long*>(vp - 3 + 4 * e) = vq[e];
        } else if (in_quad == 4 || last) {     // a quad this walk holds in part
          const int k = min(in_quad, vn);
          for (int i = 0; i < k; ++i)
#pragma unroll
            for (int e = 0; e < 8; ++e) vp[4 * e - i] = (bf16_t)(vq[e] >> (48 - 16 * i));
        }
      }
    }
  });
}

static bool conv_ok(const ConvArgs& a, int nseq) {
  return a.C > 0 && a.taps >= 1 && a.taps <= 32 && (a.taps == 1 || a.state) && a.slots &&
         (a.tiles == nullptr || a.tile >= a.taps - 1) && nseq > 0;
}

#define LMX_TAPS(F, ...)                       \
  switch (a.taps) {                            \
    case 2: F(__VA_ARGS__, 2); break;          \
    case 3: F(__VA_ARGS__, 3); break;          \
    case 4: F(__VA_ARGS__, 4); break;          \
    default: F(__VA_ARGS__, 0);                \
  }

int short_conv(const void* u, long u_ld, const float* w, const float* in_bias, const float* bias,
               void* state,
               const int* tiles, int ntiles, int tile, const int* cu_q, const int* ctx,
               const int* slots, int C, int taps, void* out, long out_ld, int act, int is_bf16,
               hipStream_t stream) {
  if (ntiles <= 0) return 0;
  const ConvArgs a{u, u_ld, w, in_bias, bias, state, tiles, cu_q, ctx, slots, C, taps, tile};
  if (!conv_ok(a, ntiles)) return -1;
  const bool vec = C % 8 == 0 && u_ld % 8 == 0 && out_ld % 8 == 0 &&
                   (((uintptr_t)u | (uintptr_t)out | (uintptr_t)state) & 15) == 0;
  const int V = vec ? 8 : 1;
  const dim3 grid(ntiles, (C / V + 255) / 256);
#define LMX_SC(T, VV, TP) \
  short_conv_kernel<T, VV, TP><<<grid, dim3(256), 0, stream>>>(a, out, out_ld, act)
  if (is_bf16) {
    if (vec) { LMX_TAPS(LMX_SC, bf16_t, 8) } else { LMX_SC(bf16_t, 1, 0); }
  } else {
    if (vec) { LMX_TAPS(LMX_SC, float, 8) } else { LMX_SC(float, 1, 0); }
  }
#undef LMX_SC
  return (int)hipGetLastError();
}

int conv_qkv_cache(const void* u, long u_ld, const float* w, const float* in_bias, void* state,
                   const int* tiles, int ntiles, int tile, const int* cu_q, const int* ctx, const int* state_slots,
                   int taps, void* q, long q_ld, void* kc, void* vc, const int* positions,
                   const int* slots, int Hq, int Hkv, int D, int dk, int BS, float eps, float coef,
                   float every, int is_bf16, hipStream_t stream) {
  if (ntiles <= 0) return 0;
  const int C = (Hq + 2 * Hkv) * D;
  const ConvArgs a{u, u_ld, w, in_bias, nullptr, state, tiles, cu_q, ctx, state_slots, C, taps, tile};
  // a head's D / 8 lanes reduce inside one wave: D a power of two, 8..512
  if (!conv_ok(a, ntiles) || D < 8 || D > 512 || (D & (D - 1)) || dk < 1 || dk > D || every <= 0.f)
    return -1;
  if (u_ld % 8 || q_ld % 8 || (((uintptr_t)u | (uintptr_t)q) & 15)) return -2;
  const QkvOut o{q, q_ld, kc, vc, positions, slots, Hq, Hkv, D, dk, BS, eps, coef, every};
  const dim3 grid(ntiles, (C / 8 + 255) / 256);
#define LMX_QC(T, TP) conv_qkv_cache_kernel<T, TP><<<grid, dim3(256), 0, stream>>>(a, o)
  if (is_bf16) { LMX_TAPS(LMX_QC, bf16_t) } else { LMX_TAPS(LMX_QC, float) }
#undef LMX_QC
  return (int)hipGetLastError();
}

}  // namespace lmx
