// K15: linear-attention / state-space scan.
//
// Per head, over the tokens of a sequence:
//     S_t = a_t S_{t-1} + s_t k_t v_t^T        (S is N x P, fp32)
//     o_t = S_t^T q_t + D v_t
// with q, k of N channels shared by `hpg` consecutive heads (a group), v of P
// channels per head.  The same kernels serve
//   * linear attention with a constant decay per head (a_t = decay[h], s_t = 1,
//     SiLU applied to q, k and v as they are loaded), and
//   * the state-space form: s_t = softplus(dt_t + dt_bias), a_t = exp(-exp(A_log)
//     s_t), D the skip weight.
// The state of a sequence lives in its slot of state[slots][H][N][P] between
// steps; a row range that starts at position 0 starts from the zero state
// whatever the slot holds, so slots are reused uncleared.
//
// Two forms:
//   * recurrent (decode, and every shape / dtype the other one does not
//     cover): one workgroup per (sequence, head, P tile), the state tile in
//     registers, fp32 arithmetic, token after token;
//   * chunked (bf16 prefill): 64-token chunks on 16x16x32 bf16 MFMA, the state
//     in the accumulators.  Everything that is fp32 in the definition stays
//     fp32 to within 2^-17: an fp32 operand of a product (decay-weighted
//     scores, state, decay-weighted v) enters the MFMA as the sum of two bf16
//     values, high part + remainder; q, k and v are bf16 as they come.
// Long sequences are cut into segments when the batch alone does not fill the
// chip: pass 1 computes each segment's own end state, a combine kernel chains
// them, pass 2 runs every segment from its true start state.
#include <algorithm>

#include "common.h"

namespace lmx {

// activations of the projections: bf16 rows round the result to bf16 (as the
// chunked form feeds it to the MFMA), fp32 rows keep it
template <typename T> __device__ __forceinline__ float silu_as(float x);
template <> __device__ __forceinline__ float silu_as<float>(float x) { return x / (1.f + expf(-x)); }
template <> __device__ __forceinline__ float silu_as<bf16_t>(float x) {
  return bf2f(f2bf(x / (1.f + __expf(-x))));
}

__device__ __forceinline__ float softplus_f(float x) { return x > 20.f ? x : log1pf(expf(x)); }

struct ScanArgs {
  const void *q, *k, *v;     // T rows, first head's channels
  long q_ld, k_ld, v_ld;     // row strides, elements
  const void* dt;            // T rows [.., H] or null
  long dt_ld;
  const float *dt_bias, *neg_a;   // [H]: dt form, a_t = exp(neg_a * s_t)
  const float *decay, *log_decay; // [H]: constant form
  const float* skip;         // [H] or null
  void* out;                 // T rows [.., H * P]
  long out_ld;
  float* state;              // [slots][H][N][P]
  const int *cu_q, *ctx, *slots;
  int H, N, P, hpg, act;     // act: SiLU on q, k, v
};

// ------------------------------------------------------------- recurrent ----
// grid (sequences, H, P tiles of `pt` columns), block 256 = (pt / VEC) column
// threads x kr row groups; thread (c, r) holds rows r, r + kr, ... of VEC
// columns in registers.  RPT = ceil(N / kr).
template <typename T, int VEC, int RPT>
__global__ void __launch_bounds__(256) scan_recurrent_kernel(ScanArgs a, int seq0, int pt) {
  extern __shared__ float scan_sm[];
  const int seq = seq0 + blockIdx.x, h = blockIdx.y, p0 = blockIdx.z * pt;
  const int slot = a.slots[seq];
  if (slot < 0) return;                       // padding row of a captured step
  const int N = a.N, P = a.P;
  const int ncol = pt / VEC, kr = 256 / ncol;
  const int c = threadIdx.x % ncol, r = threadIdx.x / ncol;
  const bool live = r < kr;
  const int pc = p0 + c * VEC;
  float* sq = scan_sm;                        // [N]
  float* sk = sq + N;                         // [N]
  float* sv = sk + N;                         // [pt]
  float* red = sv + pt;                       // [kr][pt]
  const int row0 = a.cu_q[seq], n = a.cu_q[seq + 1] - row0;
  const bool fresh = a.ctx[seq] == n;
  float* st = a.state + (((long)slot * a.H + h) * N) * P + pc;
  float S[RPT][VEC];
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int kk = r + i * kr;
#pragma unroll
    for (int e = 0; e < VEC; ++e) S[i][e] = 0.f;
    if (live && !fresh && kk < N && pc < P) {
      if constexpr (VEC == 4) {
        const float4 t = *reinterpret_cast<const float4*>(st + (long)kk * P);
        S[i][0] = t.x; S[i][1] = t.y; S[i][2] = t.z; S[i][3] = t.w;
      } else {
        S[i][0] = st[(long)kk * P];
      }
    }
  }
  const int g = h / a.hpg;
  const T* q = (const T*)a.q + (long)row0 * a.q_ld + (long)g * N;
  const T* k = (const T*)a.k + (long)row0 * a.k_ld + (long)g * N;
  const T* v = (const T*)a.v + (long)row0 * a.v_ld + (long)h * P;
  T* out = (T*)a.out + (long)row0 * a.out_ld + (long)h * P;
  const float skip = a.skip ? a.skip[h] : 0.f;
  for (int t = 0; t < n; ++t) {
    for (int i = threadIdx.x; i < N; i += 256) {
      const float qv = ld1(q + t * a.q_ld + i), kv = ld1(k + t * a.k_ld + i);
      sq[i] = a.act ? silu_as<T>(qv) : qv;
      sk[i] = a.act ? silu_as<T>(kv) : kv;
    }
    for (int i = threadIdx.x; i < pt; i += 256) {
      const float vv = p0 + i < P ? ld1(v + t * a.v_ld + p0 + i) : 0.f;
      sv[i] = a.act ? silu_as<T>(vv) : vv;
    }
    float s = 1.f, dec;
    if (a.dt) {
      s = softplus_f(ld1((const T*)a.dt + (long)(row0 + t) * a.dt_ld + h) + a.dt_bias[h]);
      dec = expf(a.neg_a[h] * s);
    } else {
      dec = a.decay[h];
    }
    __syncthreads();
    if (live) {
      float vs[VEC], o[VEC];
#pragma unroll
      for (int e = 0; e < VEC; ++e) { vs[e] = sv[c * VEC + e] * s; o[e] = 0.f; }
#pragma unroll
      for (int i = 0; i < RPT; ++i) {
        const int kk = r + i * kr;
        if (kk < N) {
          const float kv = sk[kk], qv = sq[kk];
#pragma unroll
          for (int e = 0; e < VEC; ++e) {
            S[i][e] = dec * S[i][e] + kv * vs[e];
            o[e] += qv * S[i][e];
          }
        }
      }
#pragma unroll
      for (int e = 0; e < VEC; ++e) red[r * pt + c * VEC + e] = o[e];
    }
    __syncthreads();
    for (int i = threadIdx.x; i < pt; i += 256) {
      if (p0 + i < P) {
        float o = 0.f;
        for (int j = 0; j < kr; ++j) o += red[j * pt + i];
        st1(out + t * a.out_ld + p0 + i, o + skip * sv[i]);
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int kk = r + i * kr;
    if (live && kk < N && pc < P) {
      if constexpr (VEC == 4) {
        *reinterpret_cast<float4*>(st + (long)kk * P) =
            make_float4(S[i][0], S[i][1], S[i][2], S[i][3]);
      } else {
        st[(long)kk * P] = S[i][0];
      }
    }
  }
}

// columns per workgroup: the largest power of two up to `want_pt` whose rows
// per thread fit the register tile (16 x 4 or 8 x 1 values)
static bool recurrent_shape(int N, int P, int want_pt, int* vec, int* pt, int* rpt) {
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

int scan_recurrent(const ScanArgs& a, int is_bf16, int seq0, int nseq, hipStream_t stream) {
  if (nseq <= 0) return 0;
  if (a.N <= 0 || a.P <= 0 || a.H <= 0 || a.hpg <= 0 || (a.dt == nullptr) == (a.decay == nullptr))
    return -1;
  // wide tiles once the batch alone fills the chip, narrow ones (more
  // workgroups) below that
  const long heads = (long)nseq * a.H;
  const int want = heads >= 512 ? 128 : heads >= 256 ? 64 : 32;
  int vec, pt, rpt;
  if (!recurrent_shape(a.N, a.P, want, &vec, &pt, &rpt)) return -2;
  const int kr = 256 / (pt / vec);
  const size_t smem = (size_t)(2 * a.N + pt + kr * pt) * sizeof(float);
  if (smem > 65536) return -3;
  const dim3 grid(nseq, a.H, (a.P + pt - 1) / pt);
#define LMX_REC(TT, V, R) \
  scan_recurrent_kernel<TT, V, R><<<grid, dim3(256), smem, stream>>>(a, seq0, pt)
#define LMX_REC_R(TT, V)                                                                     \
  if (rpt <= 2) LMX_REC(TT, V, 2); else if (rpt <= 4) LMX_REC(TT, V, 4);                      \
  else if (rpt <= 8) LMX_REC(TT, V, 8);
  if (is_bf16) {
    if (rpt > 8) LMX_REC(bf16_t, 4, 16);
    else if (vec == 4) { LMX_REC_R(bf16_t, 4) } else { LMX_REC_R(bf16_t, 1) }
  } else {
    if (rpt > 8) LMX_REC(float, 4, 16);
    else if (vec == 4) { LMX_REC_R(float, 4) } else { LMX_REC_R(float, 1) }
  }
#undef LMX_REC_R
#undef LMX_REC
  return (int)hipGetLastError();
}

// --------------------------------------------------------------- chunked ----
constexpr int SC = 64;     // tokens per chunk
constexpr int SCP = 72;    // padded row of the [.][64] LDS images (16-B aligned rows)
constexpr int SVT = 64;    // v columns per workgroup (16 per wave)

struct SegArgs {
  const int* segs;         // [nseg][4]: sequence, first row, last row (in the sequence), last-of-sequence
  float* ws;               // [nseg][H][N][P] segment states (modes 1, 2)
  float* ws_log;           // [nseg][H] log of the segment's total decay (mode 1)
};

__device__ __forceinline__ void split_bf16(float x, short& hi, short& lo) {
  const uint16_t h = f2bf(x);
  hi = (short)h;
  lo = (short)f2bf(x - bf2f(h));
}

__device__ __forceinline__ bf16x8_t frag_2x8(const bf16_t* p0, const bf16_t* p1) {
  return load_frag_2x8B(p0, p1);
}

// NK: N / 32 rounded up.  MODE 0: one segment per sequence, from and to the
// state slot; 1: segment end states only (start zero); 2: outputs from the
// chained segment states, the last segment writes the slot.
//
// LDS images (bf16): q [64][NK*32+8], k the same (later overlaid by the score
// images hi/lo [64][SCP]), k^T [NK*32][SCP], v^T [SVT][SCP]; fp32: cum[64],
// s[64], exp(cum)[64].
//
// Wave w computes the scores of query rows 16w..16w+15 and owns v columns
// 16w..16w+15 of outputs and state.  The state tile t of a wave sits in MFMA
// C layout (row = state channel 16t + 4g + r, col = v column), which is the
// B-operand layout of a product whose k index is permuted within 32: k slot
// (g, j) = channel 4g + j (j < 4) or 16 + 4g + j - 4.  q is read with the same
// permutation, so the state needs no transposition.
template <int NK, int MODE>
__global__ void __launch_bounds__(256, NK <= 4 ? 2 : 1) scan_chunk_kernel(ScanArgs a, SegArgs sg) {
  extern __shared__ __attribute__((aligned(16))) char chunk_sm[];
  constexpr int DK = NK * 32, LQ = DK + 8;
  constexpr int KBYTES = SC * LQ * 2 > 2 * SC * SCP * 2 ? SC * LQ * 2 : 2 * SC * SCP * 2;
  bf16_t* const sQ = reinterpret_cast<bf16_t*>(chunk_sm);
  bf16_t* const sK = sQ + (MODE == 1 ? 0 : SC * LQ);
  bf16_t* const sP = sK;                                   // hi [64][SCP], lo [64][SCP]
  bf16_t* const sKT = reinterpret_cast<bf16_t*>(reinterpret_cast<char*>(sK) +
                                                (MODE == 1 ? 0 : KBYTES));
  bf16_t* const sVT = sKT + DK * SCP;
  float* const cum = reinterpret_cast<float*>(sVT + SVT * SCP);
  float* const sdt = cum + SC;
  float* const ecum = sdt + SC;

  const int seg = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * SVT;
  const int seq = sg.segs[4 * seg], b = sg.segs[4 * seg + 1], e = sg.segs[4 * seg + 2];
  const bool last = sg.segs[4 * seg + 3] != 0;
  const int N = a.N, P = a.P;
  const int slot = a.slots[seq];
  const int qrow = a.cu_q[seq];
  const bool fresh = a.ctx[seq] == a.cu_q[seq + 1] - qrow;
  const long row0 = qrow + b;
  const int n = e - b;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, g = lane >> 4;
  const int vcol = v0 + wave * 16 + c;
  const bool vok = vcol < P;
  const int grp = h / a.hpg;
  const bf16_t* q = (const bf16_t*)a.q + row0 * a.q_ld + (long)grp * N;
  const bf16_t* k = (const bf16_t*)a.k + row0 * a.k_ld + (long)grp * N;
  const bf16_t* v = (const bf16_t*)a.v + row0 * a.v_ld + (long)h * P;
  const bf16_t* dt = a.dt ? (const bf16_t*)a.dt + row0 * a.dt_ld + h : nullptr;
  const float logd = a.dt ? 0.f : a.log_decay[h];
  const float bias = a.dt ? a.dt_bias[h] : 0.f, na = a.dt ? a.neg_a[h] : 0.f;
  const float skip = a.skip ? a.skip[h] : 0.f;

  // ---- state ----
  f32x4_t S[2 * NK];
  {
    const float* src = nullptr;
    if constexpr (MODE == 0) {
      if (!fresh) src = a.state + ((long)slot * a.H + h) * N * P;
    } else if constexpr (MODE == 2) {
      src = sg.ws + ((long)seg * a.H + h) * N * P;
    }
#pragma unroll
    for (int t = 0; t < 2 * NK; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int kk = 16 * t + 4 * g + r;
        S[t][r] = src && kk < N && vok ? src[(long)kk * P + vcol] : 0.f;
      }
  }

  // ---- staging: registers one chunk ahead ----
  // q / k pieces: lane group of 4 covers 64 B of a row, 16 rows per wave
  // instruction; v pieces the same over its 64 columns
  u16x8 rq[NK], rk[NK], rv[2];
  float rdt = 0.f;
  const u16x8 zero8 = {{0, 0, 0, 0, 0, 0, 0, 0}};
  const int prow = (tid >> 2), pch = tid & 3;            // 64 rows x 4 chunks per pass
  auto fetch = [&](int t0) {
    const bool ok = t0 + prow < n;
    const long r = t0 + prow;
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int ch = 8 * (pch + 4 * i);
      const bool in = ok && ch < N;
      if constexpr (MODE != 1)
        rq[i] = in ? *reinterpret_cast<const u16x8*>(q + r * a.q_ld + ch) : zero8;
      rk[i] = in ? *reinterpret_cast<const u16x8*>(k + r * a.k_ld + ch) : zero8;
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int ch = v0 + 8 * (pch + 4 * i);
      rv[i] = ok && ch < P ? *reinterpret_cast<const u16x8*>(v + r * a.v_ld + ch) : zero8;
    }
    if (dt && tid < SC) rdt = t0 + tid < n ? bf2f(dt[(long)(t0 + tid) * a.dt_ld]) : 0.f;
  };
  auto act8 = [&](u16x8& x) {
    if (a.act) {
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float f = bf2f(x.v[j]);
        x.v[j] = f2bf(f / (1.f + __expf(-f)));
      }
    }
  };

  float log_total = 0.f;
  if (n > 0) fetch(0);
  for (int t0 = 0; t0 < n; t0 += SC) {
    const int m = min(SC, n - t0);
    // ---- stage this chunk ----
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int ch = 8 * (pch + 4 * i);
      act8(rk[i]);
      if constexpr (MODE != 1) {
        act8(rq[i]);
        *reinterpret_cast<u16x8*>(sQ + prow * LQ + ch) = rq[i];
        *reinterpret_cast<u16x8*>(sK + prow * LQ + ch) = rk[i];
      }
#pragma unroll
      for (int j = 0; j < 8; ++j) sKT[(ch + j) * SCP + prow] = rk[i].v[j];
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int ch = 8 * (pch + 4 * i);
      act8(rv[i]);
#pragma unroll
      for (int j = 0; j < 8; ++j) sVT[(ch + j) * SCP + prow] = rv[i].v[j];
    }
    if (wave == 0) {
      // log decays and their prefix sum; rows past the end neither decay nor add
      float s = 1.f, la = logd;
      if (dt) { s = softplus_f(rdt + bias); la = na * s; }
      if (lane >= m) { s = 0.f; la = 0.f; }
      float x = la;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const float y = __shfl_up(x, o, 64);
        if (lane >= o) x += y;
      }
      cum[lane] = x;
      sdt[lane] = s;
      ecum[lane] = __expf(x);
    }
    __syncthreads();
    if (t0 + SC < n) fetch(t0 + SC);

    const float ctot = cum[SC - 1];
    if constexpr (MODE != 1) {
      // ---- scores of query rows 16 wave + c (transposed product: the query is
      // the MFMA column) ----
      f32x4_t sc[4];
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) sc[jt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < NK; ++ks) {
        const bf16x8_t qf = load_frag16B(sQ + (wave * 16 + c) * LQ + 32 * ks + 8 * g);
#pragma unroll
        for (int jt = 0; jt < 4; ++jt)
          if (jt <= wave)
            sc[jt] = mfma16(load_frag16B(sK + (jt * 16 + c) * LQ + 32 * ks + 8 * g), qf, sc[jt]);
      }
      const int qi = wave * 16 + c;
      const float ci = cum[qi];
      bf16x4_t ph[4], pl[4];
#pragma unroll
      for (int jt = 0; jt < 4; ++jt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int j = jt * 16 + 4 * g + r;
          const float w = j <= qi ? sc[jt][r] * __expf(ci - cum[j]) * sdt[j] : 0.f;
          short hi, lo;
          split_bf16(w, hi, lo);
          ph[jt][r] = hi;
          pl[jt][r] = lo;
        }
      __syncthreads();                       // every wave is done with k's rows
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) {
        *reinterpret_cast<bf16x4_t*>(sP + qi * SCP + jt * 16 + 4 * g) = ph[jt];
        *reinterpret_cast<bf16x4_t*>(sP + (SC + qi) * SCP + jt * 16 + 4 * g) = pl[jt];
      }
      __syncthreads();

      // ---- outputs: 64 queries x this wave's 16 columns ----
      f32x4_t o[4];
#pragma unroll
      for (int it = 0; it < 4; ++it) o[it] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < NK; ++ks) {
        bf16x8_t sh, sl;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          short hi, lo;
          split_bf16(S[2 * ks + (j >> 2)][j & 3], hi, lo);
          sh[j] = hi;
          sl[j] = lo;
        }
#pragma unroll
        for (int it = 0; it < 4; ++it) {
          const bf16_t* qr = sQ + (it * 16 + c) * LQ + 32 * ks + 4 * g;
          const bf16x8_t qf = frag_2x8(qr, qr + 16);
          o[it] = mfma16(qf, sh, o[it]);
          o[it] = mfma16(qf, sl, o[it]);
        }
      }
      const bf16x8_t vf0 = load_frag16B(sVT + (wave * 16 + c) * SCP + 8 * g);
      const bf16x8_t vf1 = load_frag16B(sVT + (wave * 16 + c) * SCP + 32 + 8 * g);
#pragma unroll
      for (int it = 0; it < 4; ++it) {
#pragma unroll
        for (int r = 0; r < 4; ++r) o[it][r] *= ecum[it * 16 + 4 * g + r];
        const bf16_t* pr = sP + (it * 16 + c) * SCP + 8 * g;
        o[it] = mfma16(load_frag16B(pr), vf0, o[it]);
        o[it] = mfma16(load_frag16B(pr + SC * SCP), vf0, o[it]);
        if (it >= 2) {
          o[it] = mfma16(load_frag16B(pr + 32), vf1, o[it]);
          o[it] = mfma16(load_frag16B(pr + SC * SCP + 32), vf1, o[it]);
        }
        const bf16x4_t xv =
            *reinterpret_cast<const bf16x4_t*>(sVT + (wave * 16 + c) * SCP + it * 16 + 4 * g);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int i = it * 16 + 4 * g + r;
          const float y = o[it][r] + skip * bf2f((uint16_t)xv[r]);
          if (i < m && vok)
            ((bf16_t*)a.out)[(row0 + t0 + i) * a.out_ld + (long)h * P + vcol] = f2bf(y);
        }
      }
    }
    // ---- state: S <- exp(ctot) S + k^T (w v),  w_j = exp(ctot - cum_j) s_j ----
    const float et = __expf(ctot);
    log_total += ctot;
    bf16x8_t wh[2], wl[2];
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      const bf16x8_t vf = load_frag16B(sVT + (wave * 16 + c) * SCP + 32 * ks + 8 * g);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int jj = 32 * ks + 8 * g + j;
        short hi, lo;
        split_bf16(bf2f((uint16_t)vf[j]) * __expf(ctot - cum[jj]) * sdt[jj], hi, lo);
        wh[ks][j] = hi;
        wl[ks][j] = lo;
      }
    }
#pragma unroll
    for (int t = 0; t < 2 * NK; ++t) {
#pragma unroll
      for (int r = 0; r < 4; ++r) S[t][r] *= et;
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        const bf16x8_t kf = load_frag16B(sKT + (t * 16 + c) * SCP + 32 * ks + 8 * g);
        S[t] = mfma16(kf, wh[ks], S[t]);
        S[t] = mfma16(kf, wl[ks], S[t]);
      }
    }
    __syncthreads();                         // the next chunk overwrites the images
  }

  float* dst = nullptr;
  if constexpr (MODE == 0) dst = a.state + ((long)slot * a.H + h) * N * P;
  if constexpr (MODE == 1) {
    dst = sg.ws + ((long)seg * a.H + h) * N * P;
    if (tid == 0 && v0 == 0) sg.ws_log[(long)seg * a.H + h] = log_total;
  }
  if constexpr (MODE == 2) {
    if (last) dst = a.state + ((long)slot * a.H + h) * N * P;
  }
  if (dst) {
#pragma unroll
    for (int t = 0; t < 2 * NK; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int kk = 16 * t + 4 * g + r;
        if (kk < N && vok) dst[(long)kk * P + vcol] = S[t][r];
      }
  }
}

// ws[seg] (own end state of a segment) -> the segment's start state, chained
// over the segments of each sequence.  grid (sequences, H, ceil(N P / 1024)),
// 4 elements per thread; first[s]..first[s+1] are the segments of sequence
// seq0 + s.
__global__ void __launch_bounds__(256) scan_combine_kernel(ScanArgs a, SegArgs sg, int seq0,
                                                           const int* __restrict__ first) {
  const int s = blockIdx.x, h = blockIdx.y, seq = seq0 + s;
  const long NP = (long)a.N * a.P;
  const bool fresh = a.ctx[seq] == a.cu_q[seq + 1] - a.cu_q[seq];
  const float* st = a.state + ((long)a.slots[seq] * a.H + h) * NP;
  const int f0 = first[s], f1 = first[s + 1];
  for (int e = 0; e < 4; ++e) {
    const long i = (long)blockIdx.z * 1024 + e * 256 + threadIdx.x;
    if (i >= NP) return;
    float x = fresh ? 0.f : st[i];
    for (int f = f0; f < f1; ++f) {
      float* p = sg.ws + ((long)f * a.H + h) * NP + i;
      const float own = f + 1 < f1 ? *p : 0.f;   // the last segment's own state is not needed
      *p = x;
      x = __expf(sg.ws_log[(long)f * a.H + h]) * x + own;
    }
  }
}

bool scan_chunk_ok(const ScanArgs& a) {
  auto al = [](const void* p, long ld) {
    return ((uintptr_t)p & 15) == 0 && ld % 8 == 0;
  };
  return a.N % 8 == 0 && a.P % 8 == 0 && a.N <= 256 && al(a.q, a.q_ld) && al(a.k, a.k_ld) &&
         al(a.v, a.v_ld);
}

template <int NK, int MODE>
static int launch_chunk(const ScanArgs& a, const SegArgs& sg, int nseg, hipStream_t stream) {
  constexpr int LQ = NK * 32 + 8;
  constexpr int KB = SC * LQ * 2 > 2 * SC * SCP * 2 ? SC * LQ * 2 : 2 * SC * SCP * 2;
  constexpr int smem = (MODE == 1 ? 0 : SC * LQ * 2 + KB) + NK * 32 * SCP * 2 + SVT * SCP * 2 +
                       3 * SC * 4;
  static_assert(smem <= 160 * 1024, "chunk images fit the LDS");
  static bool attr = false;
  if (smem > 65536 && !attr) {
    (void)hipFuncSetAttribute((const void*)scan_chunk_kernel<NK, MODE>,
                              hipFuncAttributeMaxDynamicSharedMemorySize, smem);
    attr = true;
  }
  scan_chunk_kernel<NK, MODE><<<dim3(nseg, a.H, (a.P + SVT - 1) / SVT), dim3(256), smem, stream>>>(
      a, sg);
  return (int)hipGetLastError();
}

// segs / first: see SegArgs and scan_combine_kernel.  one_pass: one segment
// per sequence (first unused).
int scan_chunked(const ScanArgs& a, const int* segs, int nseg, const int* first, int seq0, int nseq,
                 int one_pass, float* ws, float* ws_log, hipStream_t stream) {
  if (nseg <= 0) return 0;
  if (!scan_chunk_ok(a) || (a.dt == nullptr) == (a.log_decay == nullptr)) return -1;
  if (!one_pass && (!ws || !ws_log || !first)) return -2;
  const SegArgs sg{segs, ws, ws_log};
  const int nk = (a.N + 31) / 32;
#define LMX_CHUNK(MODE)                                                   \
  (nk <= 1 ? launch_chunk<1, MODE>(a, sg, nseg, stream)                   \
   : nk <= 2 ? launch_chunk<2, MODE>(a, sg, nseg, stream)                 \
   : nk <= 3 ? launch_chunk<3, MODE>(a, sg, nseg, stream)                 \
   : nk <= 4 ? launch_chunk<4, MODE>(a, sg, nseg, stream)                 \
             : launch_chunk<8, MODE>(a, sg, nseg, stream))
  if (one_pass) return LMX_CHUNK(0);
  int rc = LMX_CHUNK(1);
  if (rc) return rc;
  const long NP = (long)a.N * a.P;
  scan_combine_kernel<<<dim3(nseq, a.H, (unsigned)((NP + 1023) / 1024)), dim3(256), 0, stream>>>(
      a, sg, seq0, first);
  rc = (int)hipGetLastError();
  if (rc) return rc;
  return LMX_CHUNK(2);
#undef LMX_CHUNK
}

int linear_scan(const void* q, long q_ld, const void* k, long k_ld, const void* v, long v_ld,
                const void* dt, long dt_ld, const float* dt_bias, const float* neg_a,
                const float* decay, const float* log_decay, const float* skip, void* out,
                long out_ld, float* state, const int* cu_q, const int* ctx, const int* slots, int H,
                int N, int P, int hpg, int act, int is_bf16, int seq0, int nseq, const int* segs,
                int nseg, const int* first, int one_pass, float* ws, float* ws_log,
                hipStream_t stream) {
  ScanArgs a{q, k, v, q_ld, k_ld, v_ld, dt, dt_ld, dt_bias, neg_a, decay, log_decay, skip,
             out, out_ld, state, cu_q, ctx, slots, H, N, P, hpg, act};
  if (nseg > 0) {
    if (!is_bf16) return -4;
    return scan_chunked(a, segs, nseg, first, seq0, nseq, one_pass, ws, ws_log, stream);
  }
  return scan_recurrent(a, is_bf16, seq0, nseq, stream);
}

}  // namespace lmx
