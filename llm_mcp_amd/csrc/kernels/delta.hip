// K21: gated delta rule.
//
// Per head, over the tokens of a sequence, S an N x P matrix in fp32:
//     S <- g_t S;  u_t = beta_t (v_t - S^T k_t);  S <- S + k_t u_t^T;  o_t = S^T q_t
// with q, k of N channels shared by H / G consecutive heads, divided by their
// norms sqrt(sum + 1e-6), q also by sqrt(N); beta = sigmoid(b),
// g = exp(neg_a softplus(a + dt_bias)).  State slots as in linscan.hip.
//
// Norms, step sizes and decays never enter a bf16 operand: q and k stay as the
// convolution left them and their fp32 factors are applied to products.
//
//   delta_recurrent   decode, and every shape / dtype the chunks do not cover:
//                     one workgroup per (sequence, head, P tile), fp32.  Both
//                     products with the state are taken before its update
//                     (S^T q after it is g S^T q + (k q) u), one exchange per token
//   delta_prep        chunked (bf16 prefill), all chunks at once: per chunk of 64
//                     tokens and head, with c_t the decay from the chunk's start,
//                       A_tj = beta_t c_t/c_j (k_t k_j)  (j < t),  T = (I + A)^-1
//                       B_tj = c_t/c_j (q_t k_j)         (j <= t)
//                     T in fp32: 16 x 16 diagonal blocks by substitution, the
//                     others by fp32 MFMA
//   delta_chunk       chunk after chunk, with the start state S:
//                       U = T beta (v - c K S),  o = c Q S + B U,
//                       S <- c_end S + K^T (c_end / c U)
// Fp32 operands of bf16 MFMA products (S, T, B, U) are pairs high part +
// remainder, three products where both are (2^-16).
#include <algorithm>

#include "delta.h"
#include "scan.h"

namespace lmx {

// ------------------------------------------------------------- recurrent ----
// Threads and state tile as in scan_recurrent_kernel.
template <typename T, int VEC, int RPT>
__global__ void __launch_bounds__(256) delta_recurrent_kernel(DeltaArgs a, int pt) {
  extern __shared__ float delta_sm[];
  const int seq = blockIdx.x, h = blockIdx.y, p0 = blockIdx.z * pt;
  const int slot = a.slots[seq];
  if (slot < 0) return;                       // padding row of a captured step
  const int N = a.N, P = a.P;
  const int ncol = pt / VEC, kr = 256 / ncol;
  const int c = threadIdx.x % ncol, r = threadIdx.x / ncol;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int pc = p0 + c * VEC;
  // a wave's row groups meet by lane exchanges; what is left are `ns` partial sums
  const int wcol = max(ncol, 64), ns = 256 / wcol, sl = threadIdx.x / wcol;
  float* sq = delta_sm;                       // [N]
  float* sk = sq + N;                         // [N]
  float* sv = sk + N;                         // [pt]
  float* red = sv + pt;                       // [2][ns][pt]
  float* part = red + 2 * ns * pt;            // [4][3]
  const int row0 = a.cu_q[seq], n = a.cu_q[seq + 1] - row0;
  const bool fresh = a.ctx[seq] == n;
  float* st = a.state + (((long)slot * a.H + h) * N) * P + pc;
  float S[RPT][VEC];
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int kk = r + i * kr;
#pragma unroll
    for (int e = 0; e < VEC; ++e) S[i][e] = 0.f;
    if (!fresh && kk < N && pc < P) {
      if constexpr (VEC == 4) {
        const f32x4_t t = __builtin_nontemporal_load(reinterpret_cast<const f32x4_t*>(st + (long)kk * P));
        S[i][0] = t[0]; S[i][1] = t[1]; S[i][2] = t[2]; S[i][3] = t[3];
      } else {
        S[i][0] = st[(long)kk * P];
      }
    }
  }
  const int g = h / (a.H / a.G);
  const T* q = (const T*)a.q + (long)row0 * a.q_ld + (long)g * N;
  const T* k = (const T*)a.k + (long)row0 * a.k_ld + (long)g * N;
  const T* v = (const T*)a.v + (long)row0 * a.v_ld + (long)h * P;
  T* out = (T*)a.out + (long)row0 * a.out_ld + (long)h * P;
  const float bias = a.dt_bias[h], na = a.neg_a[h], qs = 1.f / sqrtf((float)N);
  for (int t = 0; t < n; ++t) {
    const float bt = ld1((const T*)a.b + (long)(row0 + t) * a.b_ld + h);
    const float at = ld1((const T*)a.a + (long)(row0 + t) * a.a_ld + h);
    float qq = 0.f, kk2 = 0.f, qk = 0.f;
    for (int i = threadIdx.x; i < N; i += 256) {
      const float qv = ld1(q + t * a.q_ld + i), kv = ld1(k + t * a.k_ld + i);
      sq[i] = qv;
      sk[i] = kv;
      qq += qv * qv;
      kk2 += kv * kv;
      qk += qv * kv;
    }
    for (int i = threadIdx.x; i < pt; i += 256)
      sv[i] = p0 + i < P ? ld1(v + t * a.v_ld + p0 + i) : 0.f;
    qq = wave_sum(qq);
    kk2 = wave_sum(kk2);
    qk = wave_sum(qk);
    if (lane == 0) { part[3 * wave] = qq; part[3 * wave + 1] = kk2; part[3 * wave + 2] = qk; }
    __syncthreads();
    qq = part[0] + part[3] + part[6] + part[9];
    kk2 = part[1] + part[4] + part[7] + part[10];
    qk = part[2] + part[5] + part[8] + part[11];
    const float rq = qs / sqrtf(qq + 1e-6f), rk = 1.f / sqrtf(kk2 + 1e-6f);
    const float beta = 1.f / (1.f + expf(-bt)), dec = expf(na * softplus_f(at + bias));
    float sa[VEC], so[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) sa[e] = so[e] = 0.f;
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
      const int kk = r + i * kr;
      if (kk < N) {
        const float kv = sk[kk], qv = sq[kk];
#pragma unroll
        for (int e = 0; e < VEC; ++e) { sa[e] += kv * S[i][e]; so[e] += qv * S[i][e]; }
      }
    }
    for (int m = ncol; m < 64; m <<= 1)
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        sa[e] += __shfl_xor(sa[e], m, 64);
        so[e] += __shfl_xor(so[e], m, 64);
      }
    if (threadIdx.x % wcol < ncol)
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        red[sl * pt + c * VEC + e] = sa[e];
        red[(ns + sl) * pt + c * VEC + e] = so[e];
      }
    __syncthreads();
    float u[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      float x = 0.f, o = 0.f;
      for (int j = 0; j < ns; ++j) {
        x += red[j * pt + c * VEC + e];
        o += red[(ns + j) * pt + c * VEC + e];
      }
      u[e] = beta * (sv[c * VEC + e] - dec * rk * x);
      if (r == 0 && pc + e < P)
        st1(out + t * a.out_ld + pc + e, rq * (dec * o + qk * rk * u[e]));
      u[e] *= rk;
    }
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
      const int kk = r + i * kr;
      if (kk < N) {
        const float kv = sk[kk];
#pragma unroll
        for (int e = 0; e < VEC; ++e) S[i][e] = dec * S[i][e] + kv * u[e];
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int kk = r + i * kr;
    if (kk < N && pc < P) {
      if constexpr (VEC == 4) {
        const f32x4_t t = {S[i][0], S[i][1], S[i][2], S[i][3]};
        __builtin_nontemporal_store(t, reinterpret_cast<f32x4_t*>(st + (long)kk * P));
      } else {
        st[(long)kk * P] = S[i][0];
      }
    }
  }
}

static bool delta_args_ok(const DeltaArgs& a) {
  return a.N > 0 && a.P > 0 && a.H > 0 && a.G > 0 && a.H % a.G == 0 && a.state && a.dt_bias && a.neg_a;
}

// sequences 0 .. nseq - 1
int delta_recurrent(const DeltaArgs& a, int nseq, int is_bf16, hipStream_t stream) {
  if (nseq <= 0) return 0;
  if (!delta_args_ok(a)) return -1;
  // wide tiles once the batch alone fills the chip, narrow ones below that
  const long heads = (long)nseq * a.H;
  const int want = heads >= 512 ? 128 : heads >= 256 ? 64 : 32;
  int vec, pt, rpt;
  if (!recurrent_shape(a.N, a.P, want, &vec, &pt, &rpt)) return -2;
  const int ns = 256 / std::max(pt / vec, 64);
  const size_t smem = (size_t)(2 * a.N + pt + 2 * ns * pt + 12) * sizeof(float);
  if (smem > 65536) return -3;
  const dim3 grid(nseq, a.H, (a.P + pt - 1) / pt);
#define LMX_REC(TT, V, R) \
  delta_recurrent_kernel<TT, V, R><<<grid, dim3(256), smem, stream>>>(a, pt)
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
constexpr int DC = 64;             // tokens per chunk
constexpr int DTILES = 6;          // 16 x 32 tiles of a lower triangle
constexpr int DMATS = 4 * DTILES * 512;   // T hi, T lo, B hi, B lo
constexpr int DVECS = 5 * DC;      // c rq | c rk | beta | c_end / c rk | c_end
constexpr int DTL = DC + 4;        // row of the fp32 matrices in LDS

// tile (row block it, token block pair ks <= it / 2) of a triangle.  A lane's 8
// tokens are 32 ks + 4 g + {0..3} and 32 ks + 16 + 4 g + {0..3}: where the
// accumulators of two row tiles hold them, so results feed the next product in
// place
__device__ __forceinline__ int tri_tile(int it, int ks) { return it < 2 ? it : it == 2 ? 2 + ks : 4 + ks; }

__device__ __forceinline__ f32x4_t mfma_f32(float a, float b, f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// grid (chunks, H), block 256.  The score images are overlaid by the fp32
// matrices A and T; B passes through T's place first.
template <int NK>
__global__ void __launch_bounds__(256) delta_prep_kernel(DeltaArgs a, const int* __restrict__ chunks,
                                                         bf16_t* __restrict__ mats,
                                                         float* __restrict__ vecs) {
  extern __shared__ __attribute__((aligned(16))) char prep_sm[];
  __shared__ float cum[DC], beta[DC], rk[DC], rq[DC];
  constexpr int LQ = 32 * NK + 8, NP = 4 * NK;
  bf16_t* const sK = reinterpret_cast<bf16_t*>(prep_sm);
  bf16_t* const sQ = sK + DC * LQ;
  float* const mA = reinterpret_cast<float*>(prep_sm);
  float* const mT = mA + DC * DTL;
  const int chunk = blockIdx.x, h = blockIdx.y;
  const int seq = chunks[2 * chunk], b0 = chunks[2 * chunk + 1];
  const long row0 = a.cu_q[seq] + b0;
  const int m = min(DC, a.cu_q[seq + 1] - (int)row0);
  const int N = a.N, g2 = h / (a.H / a.G);
  const int tid = threadIdx.x, lane = tid & 63, c = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const bf16_t* q = (const bf16_t*)a.q + row0 * a.q_ld + (long)g2 * N;
  const bf16_t* k = (const bf16_t*)a.k + row0 * a.k_ld + (long)g2 * N;
  const u32x4_t zero4 = {0, 0, 0, 0};
  {
    u32x4_t rkv[NK], rqv[NK];
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int it = tid + 256 * i, row = it / NP, ch = 8 * (it % NP);
      const bool on = row < m && ch < N;
      rkv[i] = on ? *reinterpret_cast<const u32x4_t*>(k + row * a.k_ld + ch) : zero4;
      rqv[i] = on ? *reinterpret_cast<const u32x4_t*>(q + row * a.q_ld + ch) : zero4;
    }
    if (wave == 0) {
      float la = 0.f, bt = 0.f;
      if (lane < m) {
        const float at = bf2f(((const bf16_t*)a.a)[(row0 + lane) * a.a_ld + h]);
        la = a.neg_a[h] * SCAN_LOG2E * softplus_f(at + a.dt_bias[h]);
        bt = 1.f / (1.f + expf(-bf2f(((const bf16_t*)a.b)[(row0 + lane) * a.b_ld + h])));
      }
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const float y = __shfl_up(la, o, 64);
        if (lane >= o) la += y;
      }
      cum[lane] = la;
      beta[lane] = bt;
    }
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int it = tid + 256 * i, row = it / NP, ch = 8 * (it % NP);
      *reinterpret_cast<u32x4_t*>(sK + row * LQ + ch) = rkv[i];
      *reinterpret_cast<u32x4_t*>(sQ + row * LQ + ch) = rqv[i];
    }
  }
  __syncthreads();
  // ---- scores of rows 16 wave .. + 15 (MFMA rows) with every earlier key ----
  f32x4_t kk[4], qk[4], qq = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) kk[jt] = qk[jt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int ks = 0; ks < NK; ++ks) {
    const bf16x8_t kf = load_frag16B(sK + (wave * 16 + c) * LQ + 32 * ks + 8 * g);
    const bf16x8_t qf = load_frag16B(sQ + (wave * 16 + c) * LQ + 32 * ks + 8 * g);
    qq = mfma16(qf, qf, qq);
#pragma unroll
    for (int jt = 0; jt < 4; ++jt)
      if (jt <= wave) {
        const bf16x8_t kj = load_frag16B(sK + (jt * 16 + c) * LQ + 32 * ks + 8 * g);
        kk[jt] = mfma16(kf, kj, kk[jt]);
        qk[jt] = mfma16(qf, kj, qk[jt]);
      }
  }
  // squared norms: the diagonal
  if (c >> 2 == g) {
    float ks2 = 0.f, qs2 = 0.f;
#pragma unroll
    for (int jt = 0; jt < 4; ++jt)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (r == (c & 3)) {
          if (jt == wave) ks2 = kk[jt][r];
          if (jt == 0) qs2 = qq[r];
        }
    rk[wave * 16 + c] = 1.f / sqrtf(ks2 + 1e-6f);
    rq[wave * 16 + c] = 1.f / sqrtf((qs2 + 1e-6f) * (float)N);
  }
  __syncthreads();
#pragma unroll
  for (int jt = 0; jt < 4; ++jt)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = wave * 16 + 4 * g + r, j = jt * 16 + c;
      const float dec = j <= t ? fast_exp2(cum[t] - cum[j]) * rk[j] : 0.f;
      mA[t * DTL + j] = j < t ? beta[t] * rk[t] * dec * kk[jt][r] : 0.f;
      mT[t * DTL + j] = j <= t ? rq[t] * dec * qk[jt][r] : 0.f;
    }
  bf16_t* const out = mats + ((long)chunk * a.H + h) * DMATS;
  auto emit = [&](int tri, int which) {
    const int it = tri < 2 ? tri : tri < 4 ? 2 : 3, ks = tri < 2 ? 0 : tri & 1;
    const float* src = mT + (16 * it + c) * DTL + 32 * ks + 4 * g;
    const f32x4_t x0 = *reinterpret_cast<const f32x4_t*>(src);
    const f32x4_t x1 = *reinterpret_cast<const f32x4_t*>(src + 16);
    u32x4_t hi, lo;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const f32x4_t& x = e < 2 ? x0 : x1;
      uint32_t p, r;
      split2(x[2 * (e & 1)], x[2 * (e & 1) + 1], p, r);
      hi[e] = p;
      lo[e] = r;
    }
    *reinterpret_cast<u32x4_t*>(out + ((2 * which) * DTILES + tri) * 512 + lane * 8) = hi;
    *reinterpret_cast<u32x4_t*>(out + ((2 * which + 1) * DTILES + tri) * 512 + lane * 8) = lo;
  };
  __syncthreads();
  emit(wave, 1);
  if (wave < 2) emit(4 + wave, 1);
  __syncthreads();
  {
#pragma unroll
    for (int jt = 1; jt < 4; ++jt)
      if (jt > wave)
#pragma unroll
        for (int r = 0; r < 4; ++r) mT[(wave * 16 + 4 * g + r) * DTL + jt * 16 + c] = 0.f;
    // diagonal block of T, one column per lane (the four lane groups agree)
    const float* A = mA + wave * 16 * DTL + wave * 16;
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float s = i == c ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < i; ++j) s -= A[i * DTL + j] * x[j];
      x[i] = s;
      if (g == 0) mT[(wave * 16 + i) * DTL + wave * 16 + c] = s;
    }
  }
  __syncthreads();
  // T_ij = -T_ii sum_k A_ik T_kj, one block diagonal after the other
#pragma unroll
  for (int d = 1; d < 4; ++d) {
    if (wave < 4 - d) {
      const int bi = wave + d, bj = wave;
      f32x4_t acc = {0.f, 0.f, 0.f, 0.f}, res = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int e = 0; e < d; ++e)
#pragma unroll
        for (int s = 0; s < 4; ++s) {
          const int kx = 16 * (bj + e) + 4 * s + g;
          acc = mfma_f32(mA[(16 * bi + c) * DTL + kx], mT[kx * DTL + 16 * bj + c], acc);
        }
#pragma unroll
      for (int s = 0; s < 4; ++s)
        res = mfma_f32(mT[(16 * bi + c) * DTL + 16 * bi + 4 * g + s], acc[s], res);
#pragma unroll
      for (int r = 0; r < 4; ++r) mT[(16 * bi + 4 * g + r) * DTL + 16 * bj + c] = -res[r];
    }
    __syncthreads();
  }
  emit(wave, 0);
  if (wave < 2) emit(4 + wave, 0);
  if (tid < DC) {
    float* w = vecs + ((long)chunk * a.H + h) * DVECS;
    const float e = fast_exp2(cum[tid]);
    w[tid] = e * rq[tid];
    w[DC + tid] = e * rk[tid];
    w[2 * DC + tid] = beta[tid];
    w[3 * DC + tid] = fast_exp2(cum[DC - 1] - cum[tid]) * rk[tid];
    w[4 * DC + tid] = fast_exp2(cum[DC - 1]);
  }
}

// fp32 accumulators of two row tiles (tokens 4 g + r, 16 + 4 g + r) as a pair of
// operand fragments
__device__ __forceinline__ void split_tiles(const f32x4_t& x, const f32x4_t& y, bf16x8_t& hi,
                                            bf16x8_t& lo) {
  u32x4_t h, l;
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const f32x4_t& t = e < 2 ? x : y;
    uint32_t p, r;
    split2(t[2 * (e & 1)], t[2 * (e & 1) + 1], p, r);
    h[e] = p;
    l[e] = r;
  }
  hi = __builtin_bit_cast(bf16x8_t, h);
  lo = __builtin_bit_cast(bf16x8_t, l);
}

// grid (sequences, H, ceil(P / (16 NV W))), block 64 W.  A wave owns 16 NV
// columns of v, u, o and the state (register layout as in scan_chunk_kernel).
template <int NK, int NV, int W>
__global__ void __launch_bounds__(64 * W, W == 8 ? 2 : 1) delta_chunk_kernel(
    DeltaArgs a, int seq0, const int* __restrict__ first, const bf16_t* __restrict__ mats,
    const float* __restrict__ vecs) {
  extern __shared__ __attribute__((aligned(16))) char delta_chunk_sm[];
  constexpr int NT = 64 * W, DK = NK * 32, LQ = DK + 8, VT = 16 * NV * W, NP = 4 * NK;
  bf16_t* const sQ = reinterpret_cast<bf16_t*>(delta_chunk_sm);
  bf16_t* const sK = sQ + DC * LQ;
  bf16_t* const sKT = sK + DC * LQ;
  bf16_t* const sVT = sKT + DK * DC;
  bf16_t* const sM = sVT + VT * DC;
  float* const sW = reinterpret_cast<float*>(sM + DMATS);

  const int seq = seq0 + blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * VT;
  const int N = a.N, P = a.P;
  const int slot = a.slots[seq];
  const long row0 = a.cu_q[seq];
  const int n = a.cu_q[seq + 1] - (int)row0;
  const bool fresh = a.ctx[seq] == n;
  const int tid = threadIdx.x, lane = tid & 63, c = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int vw = v0 + wave * 16 * NV;                      // this wave's first column
  const int g2 = h / (a.H / a.G);
  const bf16_t* q = (const bf16_t*)a.q + row0 * a.q_ld + (long)g2 * N;
  const bf16_t* k = (const bf16_t*)a.k + row0 * a.k_ld + (long)g2 * N;
  const bf16_t* v = (const bf16_t*)a.v + row0 * a.v_ld + (long)h * P;
  bf16_t* out = (bf16_t*)a.out + row0 * a.out_ld + (long)h * P;
  const long ch0 = first[blockIdx.x];
  mats += (ch0 * a.H + h) * DMATS;
  vecs += (ch0 * a.H + h) * DVECS;

  f32x4_t S[NV][2 * NK];
  auto state_io = [&](bool store, bool zero) {
    float* p = a.state + ((long)slot * a.H + h) * a.N * a.P;
    // opaque per call: the bounds masks of the load must not stay live until the store
    int N = a.N, P = a.P;
    asm volatile("" : "+s"(N), "+s"(P));
#pragma unroll
    for (int ct = 0; ct < NV; ++ct)
#pragma unroll
      for (int t = 0; t < 2 * NK; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int kk = 32 * (t >> 1) + 8 * g + 4 * (t & 1) + r, vc = vw + 16 * ct + c;
          const bool ok = kk < N && vc < P;
          if (store) {
            if (ok) p[(long)kk * P + vc] = S[ct][t][r];
          } else {
            S[ct][t][r] = ok && !zero ? p[(long)kk * P + vc] : 0.f;
          }
        }
  };
  state_io(false, fresh);

  // ---- staging, one chunk ahead in registers.  q: 16-B pieces of rows; k and
  // v: items of 4 consecutive rows x 8 channels (written transposed, 4 tokens at
  // a time); the matrices as they are ----
  constexpr int QI = (DC * NP + NT - 1) / NT, MI = DMATS / 8 / NT;
  constexpr int KITEMS = 16 * NP, ITEMS = KITEMS + 2 * VT, NI = (ITEMS + NT - 1) / NT;
  static_assert(DMATS / 8 % NT == 0 && DVECS <= 2 * NT, "whole passes");
  u32x4_t rq[QI], ri[NI][4], rm[MI];
  float rw[2];
  const u32x4_t zero4 = {0, 0, 0, 0};
  // per-thread byte offsets from wave-uniform bases (a chunk is far below 4 GB);
  // row numbers beyond every chunk where there is nothing to load
  static_assert(NT % NP == 0, "a q pass is whole rows");
  constexpr int QR = NT / NP;
  const int qc = 8 * (tid % NP), qrow = qc < N ? tid / NP : 1 << 20;
  const uint32_t qoff = (uint32_t)((tid / NP * a.q_ld + qc) * 2);
  uint32_t ioff[NI];
  int irow[NI];
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int it = tid + NT * i;
    const bool isk = wave * 64 + NT * i < KITEMS;          // wave-uniform
    const int x = isk ? it : it - KITEMS, np = isk ? NP : VT / 8;
    const int ch = 8 * (x % np) + (isk ? 0 : v0), r0 = 4 * (x / np);
    irow[i] = it < ITEMS && ch < (isk ? N : P) ? r0 : 1 << 20;
    ioff[i] = (uint32_t)((r0 * (isk ? a.k_ld : a.v_ld) + ch) * 2);
  }
  auto at = [](const void* base, uint32_t off) {
    return reinterpret_cast<const u32x4_t*>(reinterpret_cast<const char*>(base) + off);
  };
  auto fetch = [&](int t0) {
    const int left = min(n - t0, DC);
#pragma unroll
    for (int i = 0; i < QI; ++i)
      rq[i] = qrow + QR * i < left ? *at(q + (long)(t0 + QR * i) * a.q_ld, qoff) : zero4;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const bool isk = wave * 64 + NT * i < KITEMS;
      const long ld = isk ? a.k_ld : a.v_ld;
      const bf16_t* base = (isk ? k : v) + t0 * ld;
#pragma unroll
      for (int r = 0; r < 4; ++r)
        ri[i][r] = irow[i] + r < left ? *at(base + r * ld, ioff[i]) : zero4;
    }
    const bf16_t* mb = mats + (long)(t0 / DC) * a.H * DMATS;
    const float* vb = vecs + (long)(t0 / DC) * a.H * DVECS;
#pragma unroll
    for (int i = 0; i < MI; ++i) rm[i] = *at(mb + NT * i * 8, tid * 16u);
#pragma unroll
    for (int i = 0; i < 2; ++i)
      rw[i] = tid + NT * i < DVECS ? vb[tid + NT * i] : 0.f;
  };
  auto stage = [&]() {
#pragma unroll
    for (int i = 0; i < QI; ++i) {
      const int it = tid + NT * i, row = it / NP;
      if (row < DC) *reinterpret_cast<u32x4_t*>(sQ + row * LQ + 8 * (it % NP)) = rq[i];
    }
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int it = tid + NT * i;
      if (wave * 64 + NT * i >= ITEMS) continue;
      const bool isk = wave * 64 + NT * i < KITEMS;
      const int x = isk ? it : it - KITEMS, np = isk ? NP : VT / 8;
      const int pc = x % np, qd = x / np;
      bf16_t* const img = isk ? sKT : sVT;
      if (isk)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          *reinterpret_cast<u32x4_t*>(sK + (4 * qd + r) * LQ + 8 * pc) = ri[i][r];
      // k^T keeps its tokens in the order of the operand fragments (tri_tile)
      const int piece = isk ? 4 * (qd >> 3) + (qd & 3) : qd >> 1;
      const int half = isk ? (qd >> 2) & 1 : qd & 1;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const uint32_t sel = e & 1 ? 0x07060302u : 0x05040100u;
        const u32x2_t w = {__builtin_amdgcn_perm(ri[i][1][e >> 1], ri[i][0][e >> 1], sel),
                           __builtin_amdgcn_perm(ri[i][3][e >> 1], ri[i][2][e >> 1], sel)};
        *reinterpret_cast<u32x2_t*>(img + (8 * pc + e) * DC + 4 * half +
                                    8 * (piece ^ tr_swz(8 * pc + e))) = w;
      }
    }
#pragma unroll
    for (int i = 0; i < MI; ++i) *reinterpret_cast<u32x4_t*>(sM + (tid + NT * i) * 8) = rm[i];
#pragma unroll
    for (int i = 0; i < 2; ++i)
      if (tid + NT * i < DVECS) sW[tid + NT * i] = rw[i];
  };
  const f32x4_t z4 = {0.f, 0.f, 0.f, 0.f};

  if (n > 0) fetch(0);
  for (int t0 = 0; t0 < n; t0 += DC) {
    stage();
    lds_barrier();
    if (t0 + DC < n) fetch(t0 + DC);
    // ---- products with the start state: K S (row = token), (Q S)^T (row = column) ----
    f32x4_t x[NV][4], o[NV][4];
#pragma unroll
    for (int ct = 0; ct < NV; ++ct)
#pragma unroll
      for (int it = 0; it < 4; ++it) x[ct][it] = o[ct][it] = z4;
#pragma unroll
    for (int ks = 0; ks < NK; ++ks) {
      __builtin_amdgcn_sched_barrier(0);       // one k step's operands at a time
      bf16x8_t sh[NV], sl[NV];
#pragma unroll
      for (int ct = 0; ct < NV; ++ct) split_tiles(S[ct][2 * ks], S[ct][2 * ks + 1], sh[ct], sl[ct]);
      bf16x8_t kf[4], qf[4];
#pragma unroll
      for (int it = 0; it < 4; ++it) {
        kf[it] = load_frag16B(sK + (it * 16 + c) * LQ + 32 * ks + 8 * g);
        qf[it] = load_frag16B(sQ + (it * 16 + c) * LQ + 32 * ks + 8 * g);
      }
      // accumulators in turn: products of one do not follow each other
#pragma unroll
      for (int half = 0; half < 2; ++half)
#pragma unroll
        for (int ct = 0; ct < NV; ++ct)
#pragma unroll
          for (int it = 0; it < 4; ++it) {
            const bf16x8_t sf = half ? sl[ct] : sh[ct];
            x[ct][it] = mfma16(kf[it], sf, x[ct][it]);
            o[ct][it] = mfma16(sf, qf[it], o[ct][it]);
          }
    }
    __builtin_amdgcn_sched_barrier(0);
    // ---- beta (v - c K S), then U = T of it ----
    bf16x8_t rh[NV][2], rl[NV][2];
#pragma unroll
    for (int ct = 0; ct < NV; ++ct) {
      const int row = wave * 16 * NV + 16 * ct + c;
#pragma unroll
      for (int it = 0; it < 4; ++it) {
        const u32x2_t vv = *reinterpret_cast<const u32x2_t*>(
            sVT + row * DC + 4 * (g & 1) + 8 * ((2 * it + (g >> 1)) ^ tr_swz(row)));
        const f32x4_t ck = *reinterpret_cast<const f32x4_t*>(sW + DC + 16 * it + 4 * g);
        const f32x4_t bt = *reinterpret_cast<const f32x4_t*>(sW + 2 * DC + 16 * it + 4 * g);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float f = __uint_as_float(r & 1 ? vv[r >> 1] & 0xffff0000u : vv[r >> 1] << 16);
          x[ct][it][r] = bt[r] * (f - ck[r] * x[ct][it][r]);
        }
      }
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) split_tiles(x[ct][2 * ks], x[ct][2 * ks + 1], rh[ct][ks], rl[ct][ks]);
    }
    bf16x8_t mh[4], ml[4];
    auto load_mat = [&](int which, int ks) {
#pragma unroll
      for (int it = 2 * ks; it < 4; ++it) {
        const int f = tri_tile(it, ks);
        mh[it] = load_frag16B(sM + (which * DTILES + f) * 512 + lane * 8);
        ml[it] = load_frag16B(sM + ((which + 1) * DTILES + f) * 512 + lane * 8);
      }
    };
#pragma unroll
    for (int ct = 0; ct < NV; ++ct)
#pragma unroll
      for (int it = 0; it < 4; ++it) x[ct][it] = z4;
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      load_mat(0, ks);
#pragma unroll
      for (int e = 0; e < 3; ++e)
#pragma unroll
        for (int ct = 0; ct < NV; ++ct)
#pragma unroll
          for (int it = 2 * ks; it < 4; ++it)
            x[ct][it] = mfma16(e == 2 ? ml[it] : mh[it], e == 1 ? rl[ct][ks] : rh[ct][ks], x[ct][it]);
    }
    __builtin_amdgcn_sched_barrier(0);
    // ---- outputs (transposed) and c_end / c U ----
#pragma unroll
    for (int ct = 0; ct < NV; ++ct)
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) split_tiles(x[ct][2 * ks], x[ct][2 * ks + 1], rh[ct][ks], rl[ct][ks]);
#pragma unroll
    for (int it = 0; it < 4; ++it) {
      const float cq = sW[it * 16 + c];
#pragma unroll
      for (int ct = 0; ct < NV; ++ct) o[ct][it] *= cq;
    }
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      load_mat(2, ks);
#pragma unroll
      for (int e = 0; e < 3; ++e)
#pragma unroll
        for (int ct = 0; ct < NV; ++ct)
#pragma unroll
          for (int it = 2 * ks; it < 4; ++it)
            o[ct][it] = mfma16(e == 1 ? rl[ct][ks] : rh[ct][ks], e == 2 ? ml[it] : mh[it], o[ct][it]);
    }
#pragma unroll
    for (int it = 0; it < 4; ++it) {
      const int i = it * 16 + c;
      if (t0 + i < n) {
#pragma unroll
        for (int ct = 0; ct < NV; ++ct) {
          const int vc = vw + 16 * ct + 4 * g;             // P % 8 == 0: whole quads
          if (vc < P) {
            const f32x4_t& y = o[ct][it];
            const u32x2_t yw = {pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3])};
            *reinterpret_cast<u32x2_t*>(out + (long)(t0 + i) * a.out_ld + vc) = yw;
          }
        }
      }
    }
    __builtin_amdgcn_sched_barrier(0);
    // ---- state ----
#pragma unroll
    for (int ct = 0; ct < NV; ++ct) {
#pragma unroll
      for (int it = 0; it < 4; ++it)
        x[ct][it] *= *reinterpret_cast<const f32x4_t*>(sW + 3 * DC + 16 * it + 4 * g);
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) split_tiles(x[ct][2 * ks], x[ct][2 * ks + 1], rh[ct][ks], rl[ct][ks]);
    }
    const float et = sW[4 * DC];
#pragma unroll
    for (int tb = 0; tb < 2 * NK; tb += 4 < 2 * NK ? 4 : 2 * NK) {
      constexpr int TB = 4 < 2 * NK ? 4 : 2 * NK;
      __builtin_amdgcn_sched_barrier(0);
      bf16x8_t kf[TB][2];
#pragma unroll
      for (int t = 0; t < TB; ++t)
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
          const int row = 32 * ((tb + t) >> 1) + 8 * (c >> 2) + 4 * (t & 1) + (c & 3);
          kf[t][ks] = load_frag16B(sKT + row * DC + 8 * ((4 * ks + g) ^ tr_swz(row)));
        }
#pragma unroll
      for (int ct = 0; ct < NV; ++ct)
#pragma unroll
        for (int t = 0; t < TB; ++t) S[ct][tb + t] *= et;
#pragma unroll
      for (int e = 0; e < 4; ++e)
#pragma unroll
        for (int ct = 0; ct < NV; ++ct)
#pragma unroll
          for (int t = 0; t < TB; ++t)
            S[ct][tb + t] = mfma16(kf[t][e >> 1], e & 1 ? rl[ct][e >> 1] : rh[ct][e >> 1], S[ct][tb + t]);
    }
    lds_barrier();                             // the next chunk overwrites the images
  }
  state_io(true, false);
}

template <int NK>
static int launch_prep(const DeltaArgs& a, const int* chunks, int nchunks, bf16_t* mats, float* vecs,
                       hipStream_t stream) {
  constexpr int smem = std::max(2 * DC * (32 * NK + 8) * 2, 2 * DC * DTL * 4);
  static_assert(smem <= 128 * 1024, "images fit the LDS");
  static bool attr = false;
  if (smem > 65536 && !attr) {
    (void)hipFuncSetAttribute((const void*)delta_prep_kernel<NK>,
                              hipFuncAttributeMaxDynamicSharedMemorySize, smem);
    attr = true;
  }
  delta_prep_kernel<NK><<<dim3(nchunks, a.H), dim3(256), smem, stream>>>(a, chunks, mats, vecs);
  return (int)hipGetLastError();
}

template <int NK, int NV, int W>
static int launch_delta(const DeltaArgs& a, int seq0, int nseq, const int* first, const bf16_t* mats,
                        const float* vecs, hipStream_t stream) {
  constexpr int VT = 16 * NV * W;
  constexpr int smem = (2 * DC * (32 * NK + 8) + 32 * NK * DC + VT * DC + DMATS) * 2 + DVECS * 4;
  static_assert(smem <= 160 * 1024, "chunk images fit the LDS");
  static bool attr = false;
  if (!attr) {
    (void)hipFuncSetAttribute((const void*)delta_chunk_kernel<NK, NV, W>,
                              hipFuncAttributeMaxDynamicSharedMemorySize, smem);
    attr = true;
  }
  delta_chunk_kernel<NK, NV, W><<<dim3(nseq, a.H, (a.P + VT - 1) / VT), dim3(64 * W), smem, stream>>>(
      a, seq0, first, mats, vecs);
  return (int)hipGetLastError();
}

template <int NK>
static int delta_pair(const DeltaArgs& a, int seq0, int nseq, const int* chunks, int nchunks,
                      const int* first, bf16_t* mats, float* vecs, hipStream_t stream) {
  const int rc = launch_prep<NK>(a, chunks, nchunks, mats, vecs, stream);
  if (rc) return rc;
  // 128 columns per workgroup once they fill the chip, 64 (shorter steps) below
  if ((long)nseq * a.H * ((a.P + 127) / 128) >= 192 && a.P > 64)
    return launch_delta<NK, 1, 8>(a, seq0, nseq, first, mats, vecs, stream);
  return launch_delta<NK, 1, 4>(a, seq0, nseq, first, mats, vecs, stream);
}

// bf16 rows of sequences seq0 .. seq0 + nseq - 1.  chunks [nchunks][2]: sequence
// and first row (in it) of every chunk; first[s]: chunk of a sequence's start.
// mats [nchunks][H][DMATS], vecs [nchunks][H][DVECS]: workspace
int delta_chunks(const DeltaArgs& a, int seq0, int nseq, const int* chunks, int nchunks,
                 const int* first, void* mats, float* vecs, hipStream_t stream) {
  if (nseq <= 0 || nchunks <= 0) return 0;
  auto al = [](const void* p, long ld) { return ((uintptr_t)p & 15) == 0 && ld % 8 == 0; };
  if (!delta_args_ok(a) || a.N % 8 || a.P % 8 || a.N > 256 || !al(a.q, a.q_ld) || !al(a.k, a.k_ld) ||
      !al(a.v, a.v_ld) || !al(a.out, a.out_ld) || !al(mats, 0) || !vecs || !chunks || !first)
    return -1;
  const int nk = (a.N + 31) / 32;
  auto run = nk <= 1 ? delta_pair<1> : nk <= 2 ? delta_pair<2> : nk <= 4 ? delta_pair<4> : delta_pair<8>;
  return run(a, seq0, nseq, chunks, nchunks, first, (bf16_t*)mats, vecs, stream);
}

}  // namespace lmx
