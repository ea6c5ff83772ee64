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
//     s_t), D the skip weight;
//   * retention: linear attention whose q and k are rotated by their position
//     (neighbouring channels a pair) and k scaled: the recurrent form turns them
//     as it loads them, the chunked one runs on rows turned in place before;
//   * matrix memory (MEM): exponential input gates i and forget gates f (both as
//     logarithms) under a running maximum m that starts at 0,
//         m_t = max(f_t + m_{t-1}, i_t),  a_t = e^(f_t + m_{t-1} - m_t),
//         s_t = e^(i_t - m_t),  n_t = a_t n_{t-1} + s_t k_t,
//         o_t = S_t^T q_t / (max(|n_t q_t|, e^-m_t) + 1e-6);
//     with F the prefix sum of f, m_t - F_t is a running maximum of i_j - F_j, so
//     a chunk's weights e^(F_t - m_t - (F_j - i_j)) come from two vectors.
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

#include "scan.h"

namespace lmx {

// activations of the projections: bf16 rows round the result to bf16 (as the
// chunked form feeds it to the MFMA), fp32 rows keep it
template <typename T> __device__ __forceinline__ float silu_as(float x);
template <> __device__ __forceinline__ float silu_as<float>(float x) { return x / (1.f + expf(-x)); }
template <> __device__ __forceinline__ float silu_as<bf16_t>(float x) {
  return bf2f(f2bf(x / (1.f + __expf(-x))));
}

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
  const float* ang;          // [rows][nrot] cos | sin (recurrent form), or null
  int nrot;
  float k_scale;
  // matrix memory
  const void *ig, *fg;       // T rows [.., H]: gate projections
  long gate_ld;
  const float* gate_bias;    // [2][H]
  float cap, q_scale;
  float *sn, *sm;            // [slots][H][N], [slots][H]
};

// logarithms of the gates from their projections (biased): cap tanh(x / cap), and
// ln sigmoid of such a value
__device__ __forceinline__ void memory_gates(float cap, float& i, float& f) {
  i = cap * tanhf(i / cap);
  const float z = cap * tanhf(f / cap);
  f = fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
}

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
        const f32x4_t t = __builtin_nontemporal_load(reinterpret_cast<const f32x4_t*>(st + (long)kk * P));
        S[i][0] = t[0]; S[i][1] = t[1]; S[i][2] = t[2]; S[i][3] = t[3];
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
      sk[i] = (a.act ? silu_as<T>(kv) : kv) * a.k_scale;
      if (i < a.nrot) {
        const float* an = a.ang + (long)(row0 + t) * a.nrot + (i >> 1);
        const float cs = an[0], sn = i & 1 ? an[a.nrot >> 1] : -an[a.nrot >> 1];
        sq[i] = qv * cs + ld1(q + t * a.q_ld + (i ^ 1)) * sn;
        sk[i] = (kv * cs + ld1(k + t * a.k_ld + (i ^ 1)) * sn) * a.k_scale;
      }
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
        const f32x4_t t = {S[i][0], S[i][1], S[i][2], S[i][3]};
        __builtin_nontemporal_store(t, reinterpret_cast<f32x4_t*>(st + (long)kk * P));
      } else {
        st[(long)kk * P] = S[i][0];
      }
    }
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

// Matrix memory, token after token: one workgroup of BT threads per (sequence,
// head), since its columns share n and m; the columns in tiles of `pt`, each
// walking the tokens from the same n and m.  grid (sequences, H), layout of a tile
// as above.
template <typename T, int VEC, int RPT, int BT>
__global__ void __launch_bounds__(BT) memory_recurrent_kernel(ScanArgs a, int seq0, int pt) {
  extern __shared__ float scan_sm[];
  __shared__ float scratch[16];
  const int seq = seq0 + blockIdx.x, h = blockIdx.y;
  const int slot = a.slots[seq];
  if (slot < 0) return;                       // padding row of a captured step
  const int N = a.N, P = a.P, tid = threadIdx.x;
  const int ncol = pt / VEC, kr = BT / ncol;
  const int c = tid % ncol, r = tid / ncol;
  const bool live = r < kr;
  float* sq = scan_sm;                        // [N]
  float* sk = sq + N;                         // [N]
  float* sn = sk + N;                         // [N]
  float* sv = sn + N;                         // [pt]
  float* red = sv + pt;                       // [kr][pt]
  const int row0 = a.cu_q[seq], n = a.cu_q[seq + 1] - row0;
  const bool fresh = a.ctx[seq] == n;
  const long head = (long)slot * a.H + h;
  const float m0 = fresh ? 0.f : a.sm[head];
  const T* q = (const T*)a.q + (long)row0 * a.q_ld + (long)h * N;
  const T* k = (const T*)a.k + (long)row0 * a.k_ld + (long)h * N;
  const T* v = (const T*)a.v + (long)row0 * a.v_ld + (long)h * P;
  T* out = (T*)a.out + (long)row0 * a.out_ld + (long)h * P;
  float m = m0;
  for (int p0 = 0; p0 < P; p0 += pt) {
    const int pc = p0 + c * VEC;
    float* st = a.state + head * N * P + pc;
    float S[RPT][VEC];
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
      const int kk = r + i * kr;
#pragma unroll
      for (int e = 0; e < VEC; ++e) S[i][e] = 0.f;
      if (live && !fresh && kk < N && pc < P) {
        if constexpr (VEC == 4) {
          const f32x4_t t = __builtin_nontemporal_load(reinterpret_cast<const f32x4_t*>(st + (long)kk * P));
          S[i][0] = t[0]; S[i][1] = t[1]; S[i][2] = t[2]; S[i][3] = t[3];
        } else {
          S[i][0] = st[(long)kk * P];
        }
      }
    }
    // a thread's entries of n stay its own until the last tile stores them
    for (int i = tid; i < N; i += BT) sn[i] = fresh ? 0.f : a.sn[head * N + i];
    m = m0;
    for (int t = 0; t < n; ++t) {
      const long at = (row0 + t) * a.gate_ld + h;
      float ig = ld1((const T*)a.ig + at) + a.gate_bias[h];
      float f = ld1((const T*)a.fg + at) + a.gate_bias[a.H + h];
      memory_gates(a.cap, ig, f);
      const float mn = fmaxf(f + m, ig), keep = expf(f + m - mn), add = expf(ig - mn);
      m = mn;
      float dot = 0.f;
      for (int i = tid; i < N; i += BT) {
        const float qv = ld1(q + t * a.q_ld + i) * a.q_scale, kv = ld1(k + t * a.k_ld + i);
        const float x = keep * sn[i] + add * kv;
        sq[i] = qv;
        sk[i] = kv;
        sn[i] = x;
        dot += x * qv;
      }
      for (int i = tid; i < pt; i += BT) sv[i] = p0 + i < P ? ld1(v + t * a.v_ld + p0 + i) : 0.f;
      dot = block_sum(dot, scratch);          // (and a barrier)
      if (live) {
        float vs[VEC], o[VEC];
#pragma unroll
        for (int e = 0; e < VEC; ++e) { vs[e] = sv[c * VEC + e] * add; o[e] = 0.f; }
#pragma unroll
        for (int i = 0; i < RPT; ++i) {
          const int kk = r + i * kr;
          if (kk < N) {
            const float kv = sk[kk], qv = sq[kk];
#pragma unroll
            for (int e = 0; e < VEC; ++e) {
              S[i][e] = keep * S[i][e] + kv * vs[e];
              o[e] += qv * S[i][e];
            }
          }
        }
#pragma unroll
        for (int e = 0; e < VEC; ++e) red[r * pt + c * VEC + e] = o[e];
      }
      __syncthreads();
      const float inv = 1.f / (fmaxf(fabsf(dot), expf(-m)) + 1e-6f);
      for (int i = tid; i < pt; i += BT) {
        if (p0 + i < P) {
          float o = 0.f;
          for (int j = 0; j < kr; ++j) o += red[j * pt + i];
          st1(out + t * a.out_ld + p0 + i, o * inv);
        }
      }
      __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
      const int kk = r + i * kr;
      if (live && kk < N && pc < P) {
        if constexpr (VEC == 4) {
          const f32x4_t t = {S[i][0], S[i][1], S[i][2], S[i][3]};
          __builtin_nontemporal_store(t, reinterpret_cast<f32x4_t*>(st + (long)kk * P));
        } else {
          st[(long)kk * P] = S[i][0];
        }
      }
    }
  }
  for (int i = tid; i < N; i += BT) a.sn[head * N + i] = sn[i];
  if (tid == 0) a.sm[head] = m;               // read by every thread before the barriers above
}

int memory_recurrent(const ScanArgs& a, int is_bf16, int seq0, int nseq, hipStream_t stream) {
  if (nseq <= 0) return 0;
  // 256 threads once the batch alone fills the chip, 1024 (shallower tiles) below
  const int bt = (long)nseq * a.H >= 1024 ? 256 : 1024;
  const int vec = a.P % 4 == 0 ? 4 : 1;
  int pt = 16;
  while (pt < a.P && pt < 512) pt *= 2;
  for (;; pt /= 2) {
    const int kr = bt / (pt / vec);
    if (pt < 4) return -2;
    if (kr >= 1 && (a.N + kr - 1) / kr <= 16) break;
  }
  const int kr = bt / (pt / vec), rpt = (a.N + kr - 1) / kr;
  const size_t smem = (size_t)(3 * a.N + pt + kr * pt) * sizeof(float);
  if (smem > 65536) return -3;
  const dim3 grid(nseq, a.H);
#define LMX_MR(TT, V, R, B) \
  memory_recurrent_kernel<TT, V, R, B><<<grid, dim3(B), smem, stream>>>(a, seq0, pt)
#define LMX_MRR(TT, V, B)                                                          \
  if (rpt <= 2) LMX_MR(TT, V, 2, B); else if (rpt <= 4) LMX_MR(TT, V, 4, B);        \
  else if (rpt <= 8) LMX_MR(TT, V, 8, B); else LMX_MR(TT, V, 16, B);
#define LMX_MRB(TT, V) if (bt == 256) { LMX_MRR(TT, V, 256) } else { LMX_MRR(TT, V, 1024) }
  if (is_bf16) {
    if (vec == 4) { LMX_MRB(bf16_t, 4) } else { LMX_MRB(bf16_t, 1) }
  } else {
    if (vec == 4) { LMX_MRB(float, 4) } else { LMX_MRB(float, 1) }
  }
#undef LMX_MRB
#undef LMX_MRR
#undef LMX_MR
  return (int)hipGetLastError();
}

// --------------------------------------------------------------- chunked ----
constexpr int SC = 64;     // tokens per chunk
constexpr int SCP = 72;    // padded row of the score images (16-B aligned)
struct SegArgs {
  const int* segs;         // [nseg][4]: sequence, first row, last row (in the sequence), last-of-sequence
  float* ws;               // [nseg][H][N][P] segment states (modes 1, 2)
  float* ws_log;           // [nseg][H] log2 of the segment's total decay (mode 1)
  // MEM: [nseg][H][N + 3]: n, own m, total forget logarithm, start m (all log2)
  float* ws_n;
};

__device__ __forceinline__ float silu_fast(float x) {
  return x * __builtin_amdgcn_rcpf(1.f + fast_exp2(-x * SCAN_LOG2E));
}

__device__ __forceinline__ void silu_words(u32x4_t& w) {
#pragma unroll
  for (int m = 0; m < 4; ++m)
    w[m] = pack_bf16x2(silu_fast(__uint_as_float(w[m] << 16)),
                       silu_fast(__uint_as_float(w[m] & 0xffff0000u)));
}

// NK: N / 32 rounded up; NV: 16-column tiles per wave (a workgroup covers 64
// NV columns of v).  MODE 0: one segment per sequence, from and to the state
// slot; 1: segment end states only (start zero); 2: outputs from the chained
// segment states, the last segment writes the slot.
//
// LDS images (bf16): q [64][32 NK + 8], k the same (overlaid by the score
// images hi / lo [64][SCP] once the scores exist), k^T [32 NK][64] and v^T
// [64 NV][64] swizzled; fp32 per token: log2 decay prefix, s, 2^prefix, and
// the weight of the token in the end state.
//
// Wave w computes the scores of query rows 16w..16w+15 and owns 16 NV columns
// of outputs and state.  A state tile pair (2 ks, 2 ks + 1) keeps channels
// 32 ks + 8 g + j in lane group g (tile j >> 2, register j & 3) of its column:
// that is the operand layout of the products with q, so the state is split
// into bf16 pairs in place, with no exchange.  Outputs are computed transposed
// (MFMA row = v column): a lane ends up with 4 consecutive columns of a row.
//
// MEM: matrix memory.  cum holds F_t - m_t and sdt F_j - i_j (log2), ecum the factor
// e^(F_t + m_0 - m_t) of the chunk's start state; n is a vector in LDS that the
// first waves advance, n q is taken from the query fragments and the row sums of
// the scores.  The workgroup of the first columns writes n and m back, so where
// there are several the sequence must not run in mode 0.
template <int NK, int NV, int MODE, bool MEM = false>
__global__ void __launch_bounds__(256, NK <= 4 ? 2 : 1) scan_chunk_kernel(ScanArgs a, SegArgs sg) {
  extern __shared__ __attribute__((aligned(16))) char chunk_sm[];
  constexpr int DK = NK * 32, LQ = DK + 8, VT = 64 * NV, NP = 4 * NK;
  constexpr int KEL = MODE == 1 ? 0 : (SC * LQ > 2 * SC * SCP ? SC * LQ : 2 * SC * SCP);
  bf16_t* const sQ = reinterpret_cast<bf16_t*>(chunk_sm);
  bf16_t* const sK = sQ + (MODE == 1 ? 0 : SC * LQ);
  bf16_t* const sP = sK;                                   // hi [64][SCP], lo [64][SCP]
  bf16_t* const sKT = sK + KEL;
  bf16_t* const sVT = sKT + DK * SC;
  float* const cum = reinterpret_cast<float*>(sVT + VT * SC);
  float* const sdt = cum + SC;
  float* const ecum = sdt + SC;
  float* const wend = ecum + SC;
  float* const sinv = wend + SC;           // MEM: 1 / divisor of a row
  float* const emt = sinv + SC;            // MEM: e^-m_t
  float* const nvec = emt + SC;            // MEM: n

  const int seg = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * VT;
  const int seq = sg.segs[4 * seg], b = sg.segs[4 * seg + 1], e = sg.segs[4 * seg + 2];
  const bool last = sg.segs[4 * seg + 3] != 0;
  const int N = a.N, P = a.P;
  const int slot = a.slots[seq];
  const int qrow = a.cu_q[seq];
  const bool fresh = a.ctx[seq] == a.cu_q[seq + 1] - qrow;
  const long row0 = qrow + b;
  const int n = e - b;
  const int tid = threadIdx.x, lane = tid & 63, c = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int vw = v0 + wave * 16 * NV;                      // this wave's first column
  const int grp = h / a.hpg;
  const bf16_t* q = (const bf16_t*)a.q + row0 * a.q_ld + (long)grp * N;
  const bf16_t* k = (const bf16_t*)a.k + row0 * a.k_ld + (long)grp * N;
  const bf16_t* v = (const bf16_t*)a.v + row0 * a.v_ld + (long)h * P;
  bf16_t* out = (bf16_t*)a.out + row0 * a.out_ld + (long)h * P;
  const bf16_t* dt = a.dt ? (const bf16_t*)a.dt + row0 * a.dt_ld + h : nullptr;
  const float logd = MEM || a.dt ? 0.f : a.log_decay[h] * SCAN_LOG2E;
  const float bias = a.dt ? a.dt_bias[h] : 0.f, na = a.dt ? a.neg_a[h] * SCAN_LOG2E : 0.f;
  const float skip = a.skip ? a.skip[h] : 0.f;

  // ---- state: tile t, register r = channel 32 (t / 2) + 8 g + 4 (t % 2) + r ----
  f32x4_t S[NV][2 * NK];
  auto state_io = [&](float* p, bool store, bool zero) {
    // opaque per call: the bounds masks of the load must not stay live (in
    // scalar registers, spilled) until the store
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
  {
    float* src = MODE == 2 ? sg.ws + ((long)seg * a.H + h) * N * P
                           : a.state + ((long)slot * a.H + h) * N * P;
    state_io(src, false, MODE == 1 || (MODE == 0 && fresh));
  }
  // MEM: the segment's n and (wave 0) running maximum, log2
  float* const wsn = MEM && MODE != 0 ? sg.ws_n + ((long)seg * a.H + h) * (N + 3) : nullptr;
  float* const slot_n = MEM ? a.sn + ((long)slot * a.H + h) * N : nullptr;
  float mrun = 0.f;
  if constexpr (MEM) {
    for (int i = tid; i < DK; i += 256) {
      float x = 0.f;
      if (i < N && MODE == 2) x = wsn[i];
      if (i < N && MODE == 0 && !fresh) x = slot_n[i];
      nvec[i] = x;
    }
    if (MODE == 1) mrun = -INFINITY;
    if (MODE == 2) mrun = wsn[N + 2];
    if (MODE == 0 && !fresh) mrun = a.sm[(long)slot * a.H + h] * SCAN_LOG2E;
  }

  float log_total = 0.f;

  // ---- staging, one chunk ahead in registers.  q: 16-B pieces of rows.  k and
  // v: items of 4 consecutive rows x 8 channels, so the transposed image is
  // written 4 tokens (8 B) at a time ----
  constexpr int KITEMS = 16 * NP, ITEMS = KITEMS + 2 * VT, NI = (ITEMS + 255) / 256;
  u32x4_t rq[MODE == 1 ? 1 : NK], ri[NI][4];
  float rdt = 0.f, rfg = 0.f;              // MEM: both gates' projections
  const u32x4_t zero4 = {0, 0, 0, 0};
  // per-thread byte offsets from wave-uniform row bases (a chunk is far below 4 GB)
  static_assert(256 % NP == 0, "a q pass is whole rows");
  const int qr = tid / NP, qc = 8 * (tid % NP);
  const uint32_t qoff = (uint32_t)((qr * a.q_ld + qc) * 2);
  uint32_t ioff[NI];
  int irow[NI];              // first of the item's 4 rows; beyond every chunk: no item
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int it = tid + 256 * i;
    const bool isk = it < KITEMS;                          // wave-uniform
    const int x = isk ? it : it - KITEMS, np = isk ? NP : VT / 8;
    const int ch = 8 * (x % np) + (isk ? 0 : v0);
    irow[i] = it < ITEMS && ch < (isk ? N : P) ? 4 * (x / np) : 1 << 20;
    ioff[i] = (uint32_t)((4 * (x / np) * (isk ? a.k_ld : a.v_ld) + ch) * 2);
  }
  auto at = [](const void* base, uint32_t off) {
    return reinterpret_cast<const u32x4_t*>(reinterpret_cast<const char*>(base) + off);
  };
  auto fetch = [&](int t0) {
    const int left = n - t0;
    if constexpr (MODE != 1) {
      const bf16_t* base = q + (long)t0 * a.q_ld;
#pragma unroll
      for (int i = 0; i < NK; ++i)
        rq[i] = qr + (256 / NP) * i < left && qc < N
                    ? *at(base + (long)(256 / NP) * i * a.q_ld, qoff) : zero4;
    }
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const bool isk = wave * 64 + 256 * i < KITEMS;
      const long ld = isk ? a.k_ld : a.v_ld;
      const bf16_t* base = (isk ? k : v) + t0 * ld;
#pragma unroll
      for (int r = 0; r < 4; ++r)
        ri[i][r] = irow[i] + r < left ? *at(base + r * ld, ioff[i]) : zero4;
    }
    if constexpr (MEM) {
      if (tid < SC && t0 + tid < n) {
        const long at = (row0 + t0 + tid) * a.gate_ld + h;
        rdt = bf2f(((const bf16_t*)a.ig)[at]);
        rfg = bf2f(((const bf16_t*)a.fg)[at]);
      }
    } else {
      if (dt && tid < SC) rdt = t0 + tid < n ? bf2f(dt[(long)(t0 + tid) * a.dt_ld]) : 0.f;
    }
  };
  auto stage = [&](int m) {
    if constexpr (MODE != 1) {
#pragma unroll
      for (int i = 0; i < NK; ++i) {
        const int it = tid + 256 * i;
        if (a.act) silu_words(rq[i]);
        *reinterpret_cast<u32x4_t*>(sQ + (it / NP) * LQ + qc) = rq[i];
      }
    }
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int it = tid + 256 * i;
      if (wave * 64 + 256 * i >= ITEMS) continue;
      const bool isk = wave * 64 + 256 * i < KITEMS;
      const int x = isk ? it : it - KITEMS, np = isk ? NP : VT / 8;
      const int pc = x % np, qd = x / np;
      bf16_t* const img = isk ? sKT : sVT;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        if (a.act) silu_words(ri[i][r]);
        if constexpr (MODE != 1)
          if (isk) *reinterpret_cast<u32x4_t*>(sK + (4 * qd + r) * LQ + 8 * pc) = ri[i][r];
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        // tr_swz(8 pc + e) = swz(pc) ^ (e & 3): 4 addresses + immediates
        const uint32_t sel = e & 1 ? 0x07060302u : 0x05040100u;
        const u32x2_t w = {__builtin_amdgcn_perm(ri[i][1][e >> 1], ri[i][0][e >> 1], sel),
                           __builtin_amdgcn_perm(ri[i][3][e >> 1], ri[i][2][e >> 1], sel)};
        *reinterpret_cast<u32x2_t*>(img + 8 * pc * SC + 4 * (qd & 1) +
                                    8 * (((qd >> 1) ^ tr_swz(8 * pc)) ^ (e & 3)) + e * SC) = w;
      }
    }
    if (MEM && wave == 0) {
      __builtin_amdgcn_sched_barrier(0);
      float ig = rdt + a.gate_bias[h], f = rfg + a.gate_bias[a.H + h];
      memory_gates(a.cap, ig, f);
      f = lane < m ? f * SCAN_LOG2E : 0.f;       // rows past the end neither decay nor add
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const float y = __shfl_up(f, o, 64);
        if (lane >= o) f += y;
      }
      const float b = lane < m ? f - ig * SCAN_LOG2E : INFINITY;
      float mx = fmaxf(mrun, -b);
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const float y = __shfl_up(mx, o, 64);
        if (lane >= o) mx = fmaxf(mx, y);
      }
      const float mt = f + mx, fend = __shfl(f, 63, 64), mend = __shfl(mt, 63, 64);
      cum[lane] = f - mt;
      sdt[lane] = b;
      ecum[lane] = fast_exp2(f + mrun - mt);
      wend[lane] = fast_exp2(fend - mend - b);
      emt[lane] = fast_exp2(-mt);
      mrun = mend;
      log_total += fend;
    } else if (!MEM && wave == 0) {
      // log2 decays and their prefix sum; rows past the end neither decay nor add
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
      ecum[lane] = fast_exp2(x);
      wend[lane] = fast_exp2(__shfl(x, 63, 64) - x) * s;
    }
  };

  // k^T fragment addresses: row 32 tt + 8 (c / 4) + 4 b + c % 4, piece 4 ks + g:
  // the swizzle leaves 4 lane offsets (index tt ^ 2 ks), the rest is immediate
  const bf16_t* ktp[4];
#pragma unroll
  for (int z = 0; z < 4; ++z) {
    const int row = 8 * (c >> 2) + (c & 3);
    ktp[z] = sKT + row * SC + 8 * (g ^ tr_swz(row) ^ (2 * z));
  }

  if (n > 0) fetch(0);
  for (int t0 = 0; t0 < n; t0 += SC) {
    const int m = min(SC, n - t0);
    stage(m);
    lds_barrier();
    if (t0 + SC < n) fetch(t0 + SC);

    bf16x8_t vf[NV][2];        // v^T fragments of this wave's columns
    auto load_v = [&]() {
#pragma unroll
      for (int ct = 0; ct < NV; ++ct) {
        const int row = wave * 16 * NV + 16 * ct + c;
#pragma unroll
        for (int ks = 0; ks < 2; ++ks)
          vf[ct][ks] = load_frag16B(sVT + row * SC + 8 * ((4 * ks + g) ^ tr_swz(row)));
      }
    };
    if constexpr (MODE == 1) load_v();
    if constexpr (MODE != 1) {
      // ---- scores of query rows 16 wave + c (the query is the MFMA column) ----
      f32x4_t sc[4];
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) sc[jt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      float nq = 0.f;                      // MEM: n q, this lane's channels
#pragma unroll
      for (int ks = 0; ks < NK; ++ks) {
        __builtin_amdgcn_sched_barrier(0);
        const bf16x8_t qf = load_frag16B(sQ + (wave * 16 + c) * LQ + 32 * ks + 8 * g);
        if constexpr (MEM) {
          float nv[8];
          ldv<8>(nv, nvec + 32 * ks + 8 * g);
#pragma unroll
          for (int e = 0; e < 8; ++e) nq += nv[e] * bf2f((uint16_t)qf[e]);
        }
#pragma unroll
        for (int jt = 0; jt < 4; ++jt)
          if (jt <= wave)
            sc[jt] = mfma16(load_frag16B(sK + (jt * 16 + c) * LQ + 32 * ks + 8 * g), qf, sc[jt]);
      }
      const int qi = wave * 16 + c;
      const float ci = cum[qi];
      float rows = 0.f;                    // MEM: row sum of the scores, this lane's keys
      u32x2_t ph[4], pl[4];
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) {
        const f32x4_t cj = *reinterpret_cast<const f32x4_t*>(cum + jt * 16 + 4 * g);
        const f32x4_t sj = *reinterpret_cast<const f32x4_t*>(sdt + jt * 16 + 4 * g);
        float w[4];
        // visible keys of this tile: all, up to the query's own, or none (opaque:
        // the comparison masks are loop-invariant and would fill the scalar file)
        int lim = jt < wave ? 64 : jt == wave ? c : -1;
        asm volatile("" : "+v"(lim));
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          if constexpr (MEM) {
            w[r] = 4 * g + r <= lim ? sc[jt][r] * fast_exp2(ci - sj[r]) : 0.f;
            rows += w[r];
          } else {
            w[r] = 4 * g + r <= lim ? sc[jt][r] * fast_exp2(ci - cj[r]) * sj[r] : 0.f;
            // the skip term is a score of one's own v
            if (jt == wave) w[r] += 4 * g + r == c ? skip : 0.f;
          }
        }
        uint32_t h0, l0, h1, l1;
        split2(w[0], w[1], h0, l0);
        split2(w[2], w[3], h1, l1);
        ph[jt] = u32x2_t{h0, h1};
        pl[jt] = u32x2_t{l0, l1};
      }
      if constexpr (MEM) {
        float x = rows + ecum[qi] * nq;
        x += __shfl_xor(x, 16, 64);
        x += __shfl_xor(x, 32, 64);
        if (g == 0) sinv[qi] = a.q_scale / (fmaxf(fabsf(x * a.q_scale), emt[qi]) + 1e-6f);
      }
      lds_barrier();                       // every wave is done with k's rows
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) {
        *reinterpret_cast<u32x2_t*>(sP + qi * SCP + jt * 16 + 4 * g) = ph[jt];
        *reinterpret_cast<u32x2_t*>(sP + (SC + qi) * SCP + jt * 16 + 4 * g) = pl[jt];
      }

      // ---- outputs, transposed: state part 2^cum (S^T q) ----
      f32x4_t o[NV][4];
#pragma unroll
      for (int ct = 0; ct < NV; ++ct)
#pragma unroll
        for (int it = 0; it < 4; ++it) o[ct][it] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < NK; ++ks) {
        __builtin_amdgcn_sched_barrier(0);   // one k step's operands at a time
        bf16x8_t sh[NV], sl[NV];
#pragma unroll
        for (int ct = 0; ct < NV; ++ct) {
          u32x4_t hi, lo;
#pragma unroll
          for (int m2 = 0; m2 < 4; ++m2) {
            uint32_t x, y;
            const f32x4_t& t = S[ct][2 * ks + (m2 >> 1)];
            split2(t[2 * (m2 & 1)], t[2 * (m2 & 1) + 1], x, y);
            hi[m2] = x;
            lo[m2] = y;
          }
          sh[ct] = __builtin_bit_cast(bf16x8_t, hi);
          sl[ct] = __builtin_bit_cast(bf16x8_t, lo);
        }
#pragma unroll
        for (int it = 0; it < 4; ++it) {
          const bf16x8_t qf = load_frag16B(sQ + (it * 16 + c) * LQ + 32 * ks + 8 * g);
#pragma unroll
          for (int ct = 0; ct < NV; ++ct) {
            o[ct][it] = mfma16(sh[ct], qf, o[ct][it]);
            o[ct][it] = mfma16(sl[ct], qf, o[ct][it]);
          }
        }
      }
      load_v();
      lds_barrier();                       // the scores of every query are in LDS
#pragma unroll
      for (int it = 0; it < 4; ++it) {
        __builtin_amdgcn_sched_barrier(0);
        const int i = it * 16 + c;
        const float ec = ecum[i];
#pragma unroll
        for (int ct = 0; ct < NV; ++ct) o[ct][it] *= ec;
#pragma unroll
        for (int ks = 0; ks <= it / 2; ++ks) {
          const bf16_t* pr = sP + i * SCP + 32 * ks + 8 * g;
          const bf16x8_t pfh = load_frag16B(pr), pfl = load_frag16B(pr + SC * SCP);
#pragma unroll
          for (int ct = 0; ct < NV; ++ct) {
            o[ct][it] = mfma16(vf[ct][ks], pfh, o[ct][it]);
            o[ct][it] = mfma16(vf[ct][ks], pfl, o[ct][it]);
          }
        }
        if (i < m) {
          const float inv = MEM ? sinv[i] : 1.f;
#pragma unroll
          for (int ct = 0; ct < NV; ++ct) {
            const int vc = vw + 16 * ct + 4 * g;           // P % 8 == 0: whole quads
            if (vc < P) {
              f32x4_t y = o[ct][it];
              if constexpr (MEM) y *= inv;
              const u32x2_t yw = {pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3])};
              *reinterpret_cast<u32x2_t*>(out + (long)(t0 + i) * a.out_ld + vc) = yw;
            }
          }
        }
      }
    }
    // ---- state: S <- 2^ctot S + k^T (w v) ----
    const float ctot = cum[SC - 1], et = ecum[SC - 1];
    if constexpr (!MEM) log_total += ctot;
    if constexpr (MEM) {                   // n <- 2^.. n + k^T wend, a channel per thread
      for (int ch = tid; ch < DK; ch += 256) {
        float x = et * nvec[ch];
#pragma unroll
        for (int pc = 0; pc < 8; ++pc) {
          float kv[8], wv[8];
          ldv<8>(kv, sKT + ch * SC + 8 * (pc ^ tr_swz(ch)));
          ldv<8>(wv, wend + 8 * pc);
#pragma unroll
          for (int e = 0; e < 8; ++e) x += kv[e] * wv[e];
        }
        nvec[ch] = x;
      }
    }
    bf16x8_t wh[NV][2], wl[NV][2];
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      const f32x4_t w0 = *reinterpret_cast<const f32x4_t*>(wend + 32 * ks + 8 * g);
      const f32x4_t w1 = *reinterpret_cast<const f32x4_t*>(wend + 32 * ks + 8 * g + 4);
#pragma unroll
      for (int ct = 0; ct < NV; ++ct) {
        const u32x4_t x = __builtin_bit_cast(u32x4_t, vf[ct][ks]);
        u32x4_t hi, lo;
#pragma unroll
        for (int m2 = 0; m2 < 4; ++m2) {
          const f32x4_t& w = m2 < 2 ? w0 : w1;
          uint32_t xh, xl;
          split2(__uint_as_float(x[m2] << 16) * w[2 * (m2 & 1)],
                 __uint_as_float(x[m2] & 0xffff0000u) * w[2 * (m2 & 1) + 1], xh, xl);
          hi[m2] = xh;
          lo[m2] = xl;
        }
        wh[ct][ks] = __builtin_bit_cast(bf16x8_t, hi);
        wl[ct][ks] = __builtin_bit_cast(bf16x8_t, lo);
      }
    }
#pragma unroll
    for (int t = 0; t < 2 * NK; ++t) {
      if (t % 2 == 0) __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int ct = 0; ct < NV; ++ct) S[ct][t] *= et;
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        const bf16x8_t kf =
            load_frag16B(ktp[((t >> 1) ^ (2 * ks)) & 3] + (32 * (t >> 1) + 4 * (t & 1)) * SC);
#pragma unroll
        for (int ct = 0; ct < NV; ++ct) {
          S[ct][t] = mfma16(kf, wh[ct][ks], S[ct][t]);
          S[ct][t] = mfma16(kf, wl[ct][ks], S[ct][t]);
        }
      }
    }
    lds_barrier();                         // the next chunk overwrites the images
  }

  if constexpr (MODE == 1) {
    state_io(sg.ws + ((long)seg * a.H + h) * N * P, true, false);
    if (!MEM && tid == 0 && v0 == 0) sg.ws_log[(long)seg * a.H + h] = log_total;
  } else {
    if (MODE == 0 || last) state_io(a.state + ((long)slot * a.H + h) * N * P, true, false);
  }
  if constexpr (MEM) {
    if (v0 == 0) {
      float* const dst = MODE == 1 ? wsn : slot_n;
      if (MODE != 2 || last)
        for (int i = tid; i < N; i += 256) dst[i] = nvec[i];
      if (tid == 0) {
        if (MODE == 1) { wsn[N] = mrun; wsn[N + 1] = log_total; }
        else if (MODE == 0 || last) a.sm[(long)slot * a.H + h] = mrun / SCAN_LOG2E;
      }
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
      x = fast_exp2(sg.ws_log[(long)f * a.H + h]) * x + own;
    }
  }
}

// The same for matrix memories: segments chain under their running maxima.  grid
// (sequences, H, ceil((N P + N) / 1024)).
__global__ void __launch_bounds__(256) memory_combine_kernel(ScanArgs a, SegArgs sg, int seq0,
                                                             const int* __restrict__ first) {
  const int s = blockIdx.x, h = blockIdx.y, seq = seq0 + s, N = a.N;
  const long NP = (long)N * a.P, head = (long)a.slots[seq] * a.H + h;
  const bool fresh = a.ctx[seq] == a.cu_q[seq + 1] - a.cu_q[seq];
  const int f0 = first[s], f1 = first[s + 1];
  const float m0 = fresh ? 0.f : a.sm[head] * SCAN_LOG2E;
  for (int e = 0; e < 4; ++e) {
    const long i = (long)blockIdx.z * 1024 + e * 256 + threadIdx.x;
    if (i >= NP + N) return;
    float x = fresh ? 0.f : i < NP ? a.state[head * NP + i] : a.sn[head * N + i - NP], m = m0;
    for (int f = f0; f < f1; ++f) {
      float* const w = sg.ws_n + ((long)f * a.H + h) * (N + 3);
      float* const p = i < NP ? sg.ws + ((long)f * a.H + h) * NP + i : w + i - NP;
      if (i == 0) w[N + 2] = m;
      const float own = *p, mn = fmaxf(w[N + 1] + m, w[N]);
      *p = x;
      x = fast_exp2(w[N + 1] + m - mn) * x + fast_exp2(w[N] - mn) * own;
      m = mn;
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

template <int NK, int NV, int MODE, bool MEM>
static int launch_chunk_nv(const ScanArgs& a, const SegArgs& sg, int nseg, hipStream_t stream) {
  constexpr int LQ = NK * 32 + 8;
  constexpr int KEL = SC * LQ > 2 * SC * SCP ? SC * LQ : 2 * SC * SCP;
  constexpr int smem = ((MODE == 1 ? 0 : SC * LQ + KEL) + NK * 32 * SC + 64 * NV * SC) * 2 + 4 * SC * 4 + (MEM ? (2 * SC + NK * 32) * 4 : 0);
  static_assert(smem <= 160 * 1024, "chunk images fit the LDS");
  static bool attr = false;
  if (smem > 65536 && !attr) {
    (void)hipFuncSetAttribute((const void*)scan_chunk_kernel<NK, NV, MODE, MEM>,
                              hipFuncAttributeMaxDynamicSharedMemorySize, smem);
    attr = true;
  }
  scan_chunk_kernel<NK, NV, MODE, MEM>
      <<<dim3(nseg, a.H, (a.P + 64 * NV - 1) / (64 * NV)), dim3(256), smem, stream>>>(a, sg);
  return (int)hipGetLastError();
}

template <int NK, int MODE, bool MEM = false>
static int launch_chunk(const ScanArgs& a, const SegArgs& sg, int nseg, hipStream_t stream) {
  if constexpr (NK <= 4)
    if (a.P > 64) return launch_chunk_nv<NK, 2, MODE, MEM>(a, sg, nseg, stream);
  return launch_chunk_nv<NK, 1, MODE, MEM>(a, sg, nseg, stream);
}

// segs / first: see SegArgs and scan_combine_kernel.  one_pass: one segment
// per sequence (first unused).
int scan_chunked(const ScanArgs& a, const int* segs, int nseg, const int* first, int seq0, int nseq,
                 int one_pass, float* ws, float* ws_log, hipStream_t stream) {
  if (nseg <= 0) return 0;
  if (!scan_chunk_ok(a) || (a.dt == nullptr) == (a.log_decay == nullptr)) return -1;
  if (!one_pass && (!ws || !ws_log || !first)) return -2;
  const SegArgs sg{segs, ws, ws_log, nullptr};
  const int nk = (a.N + 31) / 32;
#define LMX_CHUNK(MODE)                                                   \
  (nk <= 1 ? launch_chunk<1, MODE>(a, sg, nseg, stream)                   \
   : nk <= 2 ? launch_chunk<2, MODE>(a, sg, nseg, stream)                 \
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

int memory_chunked(const ScanArgs& a, const int* segs, int nseg, const int* first, int seq0,
                   int nseq, int one_pass, float* ws, float* ws_n, hipStream_t stream) {
  if (nseg <= 0) return 0;
  if (!scan_chunk_ok(a)) return -1;
  // several workgroups of one head may not read and write its n and m in one pass
  if (one_pass && a.P > (a.N <= 128 ? 128 : 64)) return -6;
  if (!one_pass && (!ws || !ws_n || !first)) return -2;
  const SegArgs sg{segs, ws, nullptr, ws_n};
  const int nk = (a.N + 31) / 32;
#define LMX_CHUNK(MODE)                                                         \
  (nk <= 1 ? launch_chunk<1, MODE, true>(a, sg, nseg, stream)                   \
   : nk <= 2 ? launch_chunk<2, MODE, true>(a, sg, nseg, stream)                 \
   : nk <= 4 ? launch_chunk<4, MODE, true>(a, sg, nseg, stream)                 \
             : launch_chunk<8, MODE, true>(a, sg, nseg, stream))
  if (one_pass) return LMX_CHUNK(0);
  int rc = LMX_CHUNK(1);
  if (rc) return rc;
  const long n = (long)a.N * a.P + a.N;
  memory_combine_kernel<<<dim3(nseq, a.H, (unsigned)((n + 1023) / 1024)), dim3(256), 0, stream>>>(
      a, sg, seq0, first);
  rc = (int)hipGetLastError();
  if (rc) return rc;
  return LMX_CHUNK(2);
#undef LMX_CHUNK
}

// Rows r0..r1 - 1 of q and k (bf16, `groups` heads of N channels), in place: the
// first n channels of a head turned by the row's angles, k times k_scale.  A
// thread owns 8 channels of up to RH heads.  grid (ceil(rows N / 8 / 256),
// ceil(groups / RH), 2: q, k)
constexpr int RH = 8;
__global__ void __launch_bounds__(256) rotate_rows_kernel(bf16_t* q, long q_ld, bf16_t* k, long k_ld,
                                                          const float* __restrict__ ang, int n,
                                                          int r0, int rows, int groups, int N,
                                                          float k_scale) {
  const int np = N / 8;
  const long e0 = (long)blockIdx.x * 256 + threadIdx.x;
  if (e0 >= (long)rows * np) return;
  const long row = r0 + e0 / np;
  const int c0 = 8 * (int)(e0 % np);
  const bool isk = blockIdx.z != 0;
  const float sc = isk ? k_scale : 1.f;
  if (c0 >= n && sc == 1.f) return;
  bf16_t* base = (isk ? k + row * k_ld : q + row * q_ld) + c0;
  const int h0 = blockIdx.y * RH, h1 = min(h0 + RH, groups);
  float x[RH][8];
#pragma unroll
  for (int i = 0; i < RH; ++i)
    if (h0 + i < h1) ldv<8>(x[i], base + (long)(h0 + i) * N);
  float cs[4], sn[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const bool on = c0 + 2 * e < n;
    const float* a = ang + row * n + (c0 >> 1) + e;
    cs[e] = on ? a[0] * sc : sc;
    sn[e] = on ? a[n >> 1] * sc : 0.f;
  }
#pragma unroll
  for (int i = 0; i < RH; ++i) {
    if (h0 + i >= h1) continue;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float u = x[i][2 * e], v = x[i][2 * e + 1];
      x[i][2 * e] = u * cs[e] - v * sn[e];
      x[i][2 * e + 1] = v * cs[e] + u * sn[e];
    }
    stv<8>(base + (long)(h0 + i) * N, x[i]);
  }
}

int rotate_rows(void* q, long q_ld, void* k, long k_ld, const float* ang, int n, int r0, int r1,
                int groups, int N, float k_scale, hipStream_t stream) {
  if (r1 <= r0) return 0;
  if (groups < 1 || N < 8 || N % 8 || n < 0 || n % 2 || n > N || (n && !ang) || q_ld % 8 ||
      k_ld % 8 || (((uintptr_t)q | (uintptr_t)k) & 15))
    return -1;
  const long pieces = (long)(r1 - r0) * (N / 8);
  rotate_rows_kernel<<<dim3((unsigned)((pieces + 255) / 256), (groups + RH - 1) / RH, 2), dim3(256), 0,
                       stream>>>((bf16_t*)q, q_ld, (bf16_t*)k, k_ld, ang, n, r0, r1 - r0, groups, N,
                                 k_scale);
  return (int)hipGetLastError();
}

int linear_scan(const void* q, long q_ld, const void* k, long k_ld, const void* v, long v_ld,
                const void* dt, long dt_ld, const float* dt_bias, const float* neg_a,
                const float* decay, const float* log_decay, const float* skip, void* out,
                long out_ld, float* state, const int* cu_q, const int* ctx, const int* slots, int H,
                int N, int P, int hpg, int act, int is_bf16, const float* ang, int nrot,
                float k_scale, int seq0, int nseq, const int* segs,
                int nseg, const int* first, int one_pass, float* ws, float* ws_log,
                hipStream_t stream) {
  ScanArgs a{q, k, v, q_ld, k_ld, v_ld, dt, dt_ld, dt_bias, neg_a, decay, log_decay, skip,
             out, out_ld, state, cu_q, ctx, slots, H, N, P, hpg, act, ang, nrot, k_scale,
             nullptr, nullptr, 0, nullptr, 1.f, 1.f, nullptr, nullptr};
  if (nrot < 0 || nrot % 2 || nrot > N || (nrot && (!ang || act))) return -5;
  if (nseg > 0) {
    if (!is_bf16) return -4;
    return scan_chunked(a, segs, nseg, first, seq0, nseq, one_pass, ws, ws_log, stream);
  }
  return scan_recurrent(a, is_bf16, seq0, nseq, stream);
}

int memory_scan(const void* q, long q_ld, const void* k, long k_ld, const void* v, long v_ld,
                const void* ig, const void* fg, long gate_ld, const float* gate_bias, float cap,
                void* out, long out_ld, float* state, float* sn, float* sm, const int* cu_q,
                const int* ctx, const int* slots, int H, int N, int P, int is_bf16, int seq0,
                int nseq, const int* segs, int nseg, const int* first, int one_pass, float* ws,
                float* ws_n, hipStream_t stream) {
  if (N <= 0 || P <= 0 || H <= 0 || !ig || !fg || !gate_bias || cap <= 0.f || !sn || !sm) return -1;
  const ScanArgs a{q, k, v, q_ld, k_ld, v_ld, nullptr, 0, nullptr, nullptr, nullptr, nullptr,
                   nullptr, out, out_ld, state, cu_q, ctx, slots, H, N, P, 1, 0, nullptr, 0, 1.f,
                   ig, fg, gate_ld, gate_bias, cap, 1.f / sqrtf((float)N), sn, sm};
  if (nseg > 0) {
    if (!is_bf16) return -4;
    return memory_chunked(a, segs, nseg, first, seq0, nseq, one_pass, ws, ws_n, stream);
  }
  return memory_recurrent(a, is_bf16, seq0, nseq, stream);
}

}  // namespace lmx
