// K1: RMSNorm (+ fused residual add) and LayerNorm (+ fused residual add, for
// the post-norm nomic-bert encoder).  One workgroup per row, bf16 in/out, fp32
// statistics, 16-byte vector loads, the whole row kept in registers so the
// input is read from HBM exactly once.
//
// Replaces the normalisation Ollama/llama.cpp runs behind /api/chat and
// /api/embed (reference: worker/llm_worker/main.py:222-261,
// core/internal/api/handlers.go:1942-2015 only *call* it over HTTP).
#include "common.h"

namespace lmx {

// VPT = 8-element chunks per thread. Row length = cols, multiple of 8.
template <int VPT>
__global__ void __launch_bounds__(256) rmsnorm_kernel(
    bf16_t* __restrict__ out, bf16_t* __restrict__ residual,  // residual may be null
    const bf16_t* __restrict__ x, const bf16_t* __restrict__ w,
    int cols, long in_stride, long out_stride, float eps) {
  __shared__ float scratch[16];
  const int row = blockIdx.x;
  const bf16_t* xr = x + (long)row * in_stride;
  bf16_t* orow = out + (long)row * out_stride;
  bf16_t* rr = residual ? residual + (long)row * cols : nullptr;
  const int nchunk = cols >> 3;
  float v[VPT][8];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c < nchunk) {
      u16x8 a = *reinterpret_cast<const u16x8*>(xr + c * 8);
      if (rr) {
        u16x8 b = *reinterpret_cast<const u16x8*>(rr + c * 8);
        u16x8 h;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          // residual stream is kept in bf16 (as the model's hidden state is)
          const uint16_t hb = f2bf(bf2f(a.v[j]) + bf2f(b.v[j]));
          h.v[j] = hb;
          v[i][j] = bf2f(hb);
        }
        *reinterpret_cast<u16x8*>(rr + c * 8) = h;
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j) v[i][j] = bf2f(a.v[j]);
      }
#pragma unroll
      for (int j = 0; j < 8; ++j) ss += v[i][j] * v[i][j];
    }
  }
  // gain loads issued before the reduction: their latency overlaps it
  u16x8 wvs[VPT];
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c < nchunk) wvs[i] = *reinterpret_cast<const u16x8*>(w + c * 8);
  }
  ss = block_sum(ss, scratch);
  const float inv = rsqrtf(ss / (float)cols + eps);
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c < nchunk) {
      const u16x8 wv = wvs[i];
      u16x8 o;
#pragma unroll
      for (int j = 0; j < 8; ++j) o.v[j] = f2bf(v[i][j] * inv * bf2f(wv.v[j]));
      *reinterpret_cast<u16x8*>(orow + c * 8) = o;
    }
  }
}

// RMSNorm whose input is the S fp32 split-K partial slabs of the preceding
// projection (dgemm.hip epi 2, "partials only"): the K-split reduction, the
// residual add and the norm in one pass, so the projection needs neither a
// reduction pass nor a bf16 output round trip.  residual += sum_s slab[s]
// (rounded to bf16 once, as the bf16 hidden state), out = rms_norm(residual).
// S is a template parameter so the S x 2 slab loads of a chunk are all issued
// before the first add (a runtime trip count serialised them: S dependent
// memory latencies per chunk, ~8 us per 256-row call at S = 4).
template <int VPT, int S>
__global__ void __launch_bounds__(512) rmsnorm_slabs_kernel(
    bf16_t* __restrict__ out, bf16_t* __restrict__ residual, const float* __restrict__ slabs,
    long slab_stride, const bf16_t* __restrict__ w, int cols, long out_stride,
    float eps) {
  __shared__ float scratch[16];
  const int row = blockIdx.x;
  const float* xr = slabs + (long)row * cols;
  bf16_t* orow = out + (long)row * out_stride;
  bf16_t* rr = residual + (long)row * cols;
  const int nchunk = cols >> 3;
  float v[VPT][8];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c < nchunk) {
      f32x4_t p0[S], p1[S];
#pragma unroll
      for (int s = 0; s < S; ++s) {
        p0[s] = *reinterpret_cast<const f32x4_t*>(xr + s * slab_stride + c * 8);
        p1[s] = *reinterpret_cast<const f32x4_t*>(xr + s * slab_stride + c * 8 + 4);
      }
      const u16x8 b = *reinterpret_cast<const u16x8*>(rr + c * 8);
      f32x4_t a0 = p0[0], a1 = p1[0];
#pragma unroll
      for (int s = 1; s < S; ++s) {
        a0 += p0[s];
        a1 += p1[s];
      }
      u16x8 h;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const uint16_t hb = f2bf((j < 4 ? a0[j] : a1[j - 4]) + bf2f(b.v[j]));
        h.v[j] = hb;
        v[i][j] = bf2f(hb);
        ss += v[i][j] * v[i][j];
      }
      *reinterpret_cast<u16x8*>(rr + c * 8) = h;
    }
  }
  u16x8 wvs[VPT];
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c < nchunk) wvs[i] = *reinterpret_cast<const u16x8*>(w + c * 8);
  }
  ss = block_sum(ss, scratch);
  const float inv = rsqrtf(ss / (float)cols + eps);
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c < nchunk) {
      const u16x8 wv = wvs[i];
      u16x8 o;
#pragma unroll
      for (int j = 0; j < 8; ++j) o.v[j] = f2bf(v[i][j] * inv * bf2f(wv.v[j]));
      *reinterpret_cast<u16x8*>(orow + c * 8) = o;
    }
  }
}

template <int VPT>
__global__ void __launch_bounds__(256) layernorm_kernel(
    bf16_t* __restrict__ out, const bf16_t* __restrict__ x, const bf16_t* __restrict__ residual,
    const bf16_t* __restrict__ w, const bf16_t* __restrict__ b, int cols, float eps) {
  __shared__ float scratch[16];
  const int row = blockIdx.x;
  const bf16_t* xr = x + (long)row * cols;
  const bf16_t* rr = residual ? residual + (long)row * cols : nullptr;
  bf16_t* orow = out + (long)row * cols;
  const int nchunk = cols >> 3;
  float v[VPT][8];
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c < nchunk) {
      u16x8 a = *reinterpret_cast<const u16x8*>(xr + c * 8);
      u16x8 r;
      if (rr) r = *reinterpret_cast<const u16x8*>(rr + c * 8);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        float t = bf2f(a.v[j]);
        if (rr) t = bf2f(f2bf(t + bf2f(r.v[j])));
        v[i][j] = t;
        s += t;
      }
    }
  }
  const float mean = block_sum(s, scratch) / (float)cols;
  float sq = 0.f;
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c < nchunk) {
#pragma unroll
      for (int j = 0; j < 8; ++j) { const float d = v[i][j] - mean; sq += d * d; }
    }
  }
  const float inv = rsqrtf(block_sum(sq, scratch) / (float)cols + eps);
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c < nchunk) {
      u16x8 wv = *reinterpret_cast<const u16x8*>(w + c * 8);
      u16x8 bv = *reinterpret_cast<const u16x8*>(b + c * 8);
      u16x8 o;
#pragma unroll
      for (int j = 0; j < 8; ++j) o.v[j] = f2bf((v[i][j] - mean) * inv * bf2f(wv.v[j]) + bf2f(bv.v[j]));
      *reinterpret_cast<u16x8*>(orow + c * 8) = o;
    }
  }
}

static int pick_threads(int nchunk) {
  int t = ((nchunk + 63) / 64) * 64;
  return t > 256 ? 256 : (t < 64 ? 64 : t);
}

int rmsnorm(void* out, void* residual, const void* x, const void* w, int rows, int cols,
            long in_stride, long out_stride, float eps, hipStream_t stream) {
  if (cols % 8 != 0 || rows <= 0) return -1;
  const int nchunk = cols / 8;
  const int threads = pick_threads(nchunk);
  const int vpt = (nchunk + threads - 1) / threads;
  dim3 g(rows), b(threads);
#define LMX_RMS(V)                                                                      \
  rmsnorm_kernel<V><<<g, b, 0, stream>>>((bf16_t*)out, (bf16_t*)residual, (const bf16_t*)x, \
                                         (const bf16_t*)w, cols, in_stride, out_stride, eps)
  if (vpt <= 1) LMX_RMS(1);
  else if (vpt <= 2) LMX_RMS(2);
  else if (vpt <= 4) LMX_RMS(4);
  else if (vpt <= 8) LMX_RMS(8);
  else return -2;
#undef LMX_RMS
  return (int)hipGetLastError();
}

// Row scales of the RMSNorm folded into the projections (pgemm.hip NRM, prefill):
//   s[r] = rsqrt(sum_j part[r][j] / cols + eps)
// from the producing residual GEMM's fixed per-64-column partials (P per row,
// summed in slot order: deterministic), or -- part == null -- from the bf16
// rows of x themselves (the first layer's input: the embedding rows).
__global__ void __launch_bounds__(256) row_scale_part_kernel(float* __restrict__ s,
                                                             const float* __restrict__ part,
                                                             int M, int P, float inv_cols,
                                                             float eps) {
  const int r = blockIdx.x * 256 + threadIdx.x;
  if (r >= M) return;
  const float4* p = reinterpret_cast<const float4*>(part + (long)r * P);
  float acc = 0.f;
  for (int j = 0; j < P / 4; ++j) {
    const float4 v = p[j];
    acc += v.x;
    acc += v.y;
    acc += v.z;
    acc += v.w;
  }
  s[r] = rsqrtf(acc * inv_cols + eps);
}

template <int VPT>
__global__ void __launch_bounds__(256) row_scale_x_kernel(float* __restrict__ s,
                                                          const bf16_t* __restrict__ x,
                                                          long stride, int cols, float eps) {
  __shared__ float scratch[16];
  const bf16_t* xr = x + (long)blockIdx.x * stride;
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c < cols / 8) {
      const u16x8 a = *reinterpret_cast<const u16x8*>(xr + c * 8);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float v = bf2f(a.v[j]);
        ss += v * v;
      }
    }
  }
  ss = block_sum(ss, scratch);
  if (threadIdx.x == 0) s[blockIdx.x] = rsqrtf(ss / (float)cols + eps);
}

int row_scale(float* s, const float* part, int P, const void* x, long x_stride, int M, int cols,
              float eps, hipStream_t stream) {
  if (M <= 0) return 0;
  if (cols % 8 != 0) return -1;
  if (part) {
    if (P % 4 != 0 || P <= 0) return -1;
    row_scale_part_kernel<<<dim3((M + 255) / 256), dim3(256), 0, stream>>>(s, part, M, P,
                                                                          1.f / (float)cols, eps);
  } else {
    const int nchunk = cols / 8, threads = pick_threads(nchunk);
    const int vpt = (nchunk + threads - 1) / threads;
#define LMX_RSX(V)                                                                      \
  row_scale_x_kernel<V><<<dim3(M), dim3(threads), 0, stream>>>(s, (const bf16_t*)x, x_stride, \
                                                               cols, eps)
    if (vpt <= 1) LMX_RSX(1);
    else if (vpt <= 2) LMX_RSX(2);
    else if (vpt <= 4) LMX_RSX(4);
    else if (vpt <= 8) LMX_RSX(8);
    else return -2;
#undef LMX_RSX
  }
  return (int)hipGetLastError();
}

// workgroup cap of the slab norm (probe knob: tools/slab_norm_probe.py)
static int g_slab_threads = 512;
void set_slab_norm_threads(int t) { g_slab_threads = t < 64 ? 64 : (t > 512 ? 512 : t); }

int rmsnorm_slabs(void* out, void* residual, const float* slabs, int S, long slab_stride,
                  const void* w, int rows, int cols, long out_stride, float eps,
                  hipStream_t stream) {
  if (cols % 8 != 0 || rows <= 0 || S < 1 || residual == nullptr) return -1;
  const int nchunk = cols / 8;
  // up to 512 threads (one 8-column chunk per thread at hidden 4096): a
  // decode step has one workgroup per row (~one per CU), so the S slabs'
  // loads of a row are spread over twice the waves of the plain norm
  int threads = ((nchunk + 63) / 64) * 64;
  threads = threads > g_slab_threads ? g_slab_threads : (threads < 64 ? 64 : threads);
  const int vpt = (nchunk + threads - 1) / threads;
  dim3 g(rows), b(threads);
#define LMX_RMSS(V, SS)                                                                     \
  rmsnorm_slabs_kernel<V, SS><<<g, b, 0, stream>>>((bf16_t*)out, (bf16_t*)residual, slabs,  \
                                                   slab_stride, (const bf16_t*)w, cols,     \
                                                   out_stride, eps)
#define LMX_RMSS_S(V)                                                                       \
  switch (S) {                                                                              \
    case 1: LMX_RMSS(V, 1); break;                                                          \
    case 2: LMX_RMSS(V, 2); break;                                                          \
    case 4: LMX_RMSS(V, 4); break;                                                          \
    case 8: LMX_RMSS(V, 8); break;                                                          \
    case 16: LMX_RMSS(V, 16); break;                                                        \
    default: return -3;                                                                     \
  }
  if (vpt <= 1) { LMX_RMSS_S(1) }
  else if (vpt <= 2) { LMX_RMSS_S(2) }
  else if (vpt <= 4) { LMX_RMSS_S(4) }
  else return -2;
#undef LMX_RMSS_S
#undef LMX_RMSS
  return (int)hipGetLastError();
}

int layernorm(void* out, const void* x, const void* residual, const void* w, const void* b,
              int rows, int cols, float eps, hipStream_t stream) {
  if (cols % 8 != 0 || rows <= 0) return -1;
  const int nchunk = cols / 8;
  const int threads = pick_threads(nchunk);
  const int vpt = (nchunk + threads - 1) / threads;
  dim3 g(rows), bl(threads);
#define LMX_LN(V)                                                                    \
  layernorm_kernel<V><<<g, bl, 0, stream>>>((bf16_t*)out, (const bf16_t*)x,           \
                                            (const bf16_t*)residual, (const bf16_t*)w, \
                                            (const bf16_t*)b, cols, eps)
  if (vpt <= 1) LMX_LN(1);
  else if (vpt <= 2) LMX_LN(2);
  else if (vpt <= 4) LMX_LN(4);
  else if (vpt <= 8) LMX_LN(8);
  else return -2;
#undef LMX_LN
  return (int)hipGetLastError();
}

// Sandwich norm: the norm after a sublayer, the residual add and the norm
// before the next sublayer in one pass, over an fp32 residual stream.
//
//   r   = ids ? scale * table[ids[row]] : residual[row]
//   r  += norm(y[row] + bias + own[row] r) * w_post
//                           (y: the sublayer's output, bias, own: all optional)
//   out = w_pre ? norm(r) * w_pre : r
//
// norm(x) = x / sqrt(mean(x^2) + eps); the gains are fp32 (a weight stored
// around zero arrives as 1 + w, a constant on what is added is part of w_post).
// y is T rows, S fp32 split-K slabs [S][rows][cols] summed here, or a mixture
// sum_j mix_w[row][j] y[mix_pos[row][j]] of T rows (pos -1: no such row).
// rows_idx (optional): out row i is source row
// rows_idx[i] and the residual is left as it is (the final norm of the sampled
// rows); otherwise the residual row is written when it changed.
struct SandwichArgs {
  void* out;
  float* residual;
  const void* y;
  long y_ld, slab_stride;
  int slabs;                  // 0: y is T rows
  const int* mix_pos;         // [rows][mix_n] or null
  const float* mix_w;
  int mix_n;
  const float* own;           // [rows] or null: weight of the stream's own row
  const float* bias;          // [cols] or null
  const int* ids;
  const void* table;
  float scale;
  const float *w_post, *w_pre;
  const long* rows_idx;
  int cols;
  float eps;
};

template <typename T, int V, int VPT>
__global__ void __launch_bounds__(512) sandwich_norm_kernel(SandwichArgs a) {
  __shared__ float scratch[16];
  const long src = a.rows_idx ? a.rows_idx[blockIdx.x] : blockIdx.x;
  const int cols = a.cols, nchunk = cols / V;
  float* rr = a.residual + src * cols;
  float r[VPT][V], y[VPT][V];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c >= nchunk) continue;
    if (a.ids) {
      ldv<V>(r[i], (const T*)a.table + (long)a.ids[src] * cols + c * V);
#pragma unroll
      for (int e = 0; e < V; ++e) r[i][e] *= a.scale;
    } else {
      ldv<V>(r[i], rr + c * V);
    }
    if (a.y) {
      if (a.slabs) {
        const float* p = (const float*)a.y + src * cols + c * V;
        ldv<V>(y[i], p);
        for (int s = 1; s < a.slabs; ++s) {
          float t[V];
          ldv<V>(t, p + s * a.slab_stride);
#pragma unroll
          for (int e = 0; e < V; ++e) y[i][e] += t[e];
        }
      } else if (a.mix_pos) {
#pragma unroll
        for (int e = 0; e < V; ++e) y[i][e] = 0.f;
#pragma unroll 4
        for (int j = 0; j < a.mix_n; ++j) {
          float t[V];
          const int at = a.mix_pos[src * a.mix_n + j];
          if (at < 0) continue;
          ldv<V>(t, (const T*)a.y + (long)at * a.y_ld + c * V);
          const float w = a.mix_w[src * a.mix_n + j];
#pragma unroll
          for (int e = 0; e < V; ++e) y[i][e] += w * t[e];
        }
      } else {
        ldv<V>(y[i], (const T*)a.y + src * a.y_ld + c * V);
      }
      if (a.own) {
        const float w = a.own[src];
#pragma unroll
        for (int e = 0; e < V; ++e) y[i][e] += w * r[i][e];
      }
      if (a.bias) {
        float t[V];
        ldv<V>(t, a.bias + c * V);
#pragma unroll
        for (int e = 0; e < V; ++e) y[i][e] += t[e];
      }
#pragma unroll
      for (int e = 0; e < V; ++e) ss += y[i][e] * y[i][e];
    }
  }
  if (a.y) {
    ss = block_sum(ss, scratch);
    const float inv = rsqrtf(ss / (float)cols + a.eps);
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      const int c = threadIdx.x + i * blockDim.x;
      if (c >= nchunk) continue;
      float w[V];
      ldv<V>(w, a.w_post + c * V);
#pragma unroll
      for (int e = 0; e < V; ++e) r[i][e] += y[i][e] * inv * w[e];
    }
  }
  if (!a.rows_idx && (a.y || a.ids)) {
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      const int c = threadIdx.x + i * blockDim.x;
      if (c < nchunk) stv<V>(rr + c * V, r[i]);
    }
  }
  if (!a.w_pre) {
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      const int c = threadIdx.x + i * blockDim.x;
      if (c < nchunk) stv<V>((T*)a.out + (long)blockIdx.x * cols + c * V, r[i]);
    }
    return;
  }
  ss = 0.f;
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c < nchunk)
#pragma unroll
      for (int e = 0; e < V; ++e) ss += r[i][e] * r[i][e];
  }
  ss = block_sum(ss, scratch);
  const float inv = rsqrtf(ss / (float)cols + a.eps);
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c >= nchunk) continue;
    float w[V];
    ldv<V>(w, a.w_pre + c * V);
#pragma unroll
    for (int e = 0; e < V; ++e) w[e] *= r[i][e] * inv;
    stv<V>((T*)a.out + (long)blockIdx.x * cols + c * V, w);
  }
}

int sandwich_norm(void* out, float* residual, const void* y, long y_ld, int slabs, long slab_stride,
                  const int* mix_pos, const float* mix_w, int mix_n, const float* own,
                  const float* bias, const int* ids,
                  const void* table, float scale, const float* w_post, const float* w_pre,
                  const long* rows_idx, int rows, int cols, float eps, int is_bf16,
                  hipStream_t stream) {
  if (rows <= 0) return 0;
  if (cols <= 0 || !residual || !out || (y && !w_post) || (mix_pos && (!y || !mix_w || slabs)) ||
      ((own || bias) && !y))
    return -1;
  const SandwichArgs a{out, residual, y, y_ld, slab_stride, slabs, mix_pos, mix_w, mix_n, own,
                       bias, ids, table, scale, w_post, w_pre, rows_idx, cols, eps};
  const bool vec = cols % 8 == 0 && y_ld % 8 == 0;
  const int nchunk = vec ? cols / 8 : cols;
  const int vpt = (nchunk + 511) / 512;
  if (vpt > (vec ? 4 : 8)) return -2;
  const int threads = nchunk >= 512 ? 512 : (nchunk + 63) / 64 * 64;
#define LMX_SW(T, V, P) sandwich_norm_kernel<T, V, P><<<dim3(rows), dim3(threads), 0, stream>>>(a)
#define LMX_SWT(T)                                                            \
  if (vec) {                                                                  \
    if (vpt == 1) LMX_SW(T, 8, 1); else if (vpt == 2) LMX_SW(T, 8, 2);        \
    else LMX_SW(T, 8, 4);                                                     \
  } else {                                                                    \
    if (vpt == 1) LMX_SW(T, 1, 1); else LMX_SW(T, 1, 8);                      \
  }
  if (is_bf16) { LMX_SWT(bf16_t) } else { LMX_SWT(float) }
#undef LMX_SWT
#undef LMX_SW
  return (int)hipGetLastError();
}

// Norm of the sum: a decoder whose residual stream (fp32) is the layer norm of
// what is added up.
//
//   r   = ln(alpha residual[row] + scale y[row]) * w_post    (residual[row] without y)
//   out = w_pre ? ln(r) * w_pre : r
//
// ln(x) = (x - mean) / sqrt(mean((x - mean)^2) + eps).  y is T rows, split-K
// slabs, a mixture of expert rows (all as in the sandwich norm), or two such
// branches, each divided by its root mean square, with a gain each.  rows_idx:
// as in the sandwich norm.
struct SubRows {
  const void* y;
  long ld, slab_stride;
  int slabs;                  // 0: T rows
};

template <typename T, int V>
__device__ __forceinline__ void load_sub(float (&f)[V], const SubRows& s, long row, int cols, int c0) {
  if (s.slabs) {
    const float* p = (const float*)s.y + row * cols + c0;
    ldv<V>(f, p);
    for (int i = 1; i < s.slabs; ++i) {
      float t[V];
      ldv<V>(t, p + i * s.slab_stride);
#pragma unroll
      for (int e = 0; e < V; ++e) f[e] += t[e];
    }
  } else {
    ldv<V>(f, (const T*)s.y + row * s.ld + c0);
  }
}

struct SumNormArgs {
  void* out;
  float* residual;
  SubRows a, b;               // b.y: the second branch, or null
  const int* mix_pos;         // [rows][mix_n] or null: a is expert rows
  const float* mix_w;
  int mix_n;
  const float *wa, *wb;       // gains of the branches
  float alpha;
  const float *scale, *w_post, *w_pre;
  const long* rows_idx;
  int cols;
  float eps;
};

template <typename T, int V, int VPT>
__global__ void __launch_bounds__(512) sum_norm_kernel(SumNormArgs a) {
  __shared__ float scratch[16];
  const long src = a.rows_idx ? a.rows_idx[blockIdx.x] : blockIdx.x;
  const int cols = a.cols, nchunk = cols / V;
  float* rr = a.residual + src * cols;
  float r[VPT][V];
  auto chunks = [&](auto&& body) {
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      const int c = threadIdx.x + i * blockDim.x;
      if (c < nchunk) body(i, c * V);
    }
  };
  auto ln = [&](const float* __restrict__ gain) {
    float s = 0.f, q = 0.f;
    chunks([&](int i, int) {
#pragma unroll
      for (int e = 0; e < V; ++e) s += r[i][e];
    });
    const float mean = block_sum(s, scratch) / (float)cols;
    chunks([&](int i, int) {
#pragma unroll
      for (int e = 0; e < V; ++e) { r[i][e] -= mean; q += r[i][e] * r[i][e]; }
    });
    const float inv = rsqrtf(block_sum(q, scratch) / (float)cols + a.eps);
    chunks([&](int i, int c0) {
      float w[V];
      ldv<V>(w, gain + c0);
#pragma unroll
      for (int e = 0; e < V; ++e) r[i][e] *= inv * w[e];
    });
  };
  chunks([&](int i, int c0) { ldv<V>(r[i], rr + c0); });
  if (a.a.y) {
    float y[VPT][V];
    if (a.mix_pos) {
      chunks([&](int i, int c0) {
#pragma unroll
        for (int e = 0; e < V; ++e) y[i][e] = 0.f;
#pragma unroll 4
        for (int j = 0; j < a.mix_n; ++j) {
          float t[V];
          ldv<V>(t, (const T*)a.a.y + (long)a.mix_pos[src * a.mix_n + j] * a.a.ld + c0);
          const float w = a.mix_w[src * a.mix_n + j];
#pragma unroll
          for (int e = 0; e < V; ++e) y[i][e] += w * t[e];
        }
      });
    } else {
      chunks([&](int i, int c0) { load_sub<T, V>(y[i], a.a, src, cols, c0); });
      if (a.b.y) {
        float z[VPT][V], sa = 0.f, sb = 0.f;
        chunks([&](int i, int c0) {
          load_sub<T, V>(z[i], a.b, src, cols, c0);
#pragma unroll
          for (int e = 0; e < V; ++e) { sa += y[i][e] * y[i][e]; sb += z[i][e] * z[i][e]; }
        });
        const float ia = rsqrtf(block_sum(sa, scratch) / (float)cols + a.eps);
        const float ib = rsqrtf(block_sum(sb, scratch) / (float)cols + a.eps);
        chunks([&](int i, int c0) {
          float wa[V], wb[V];
          ldv<V>(wa, a.wa + c0);
          ldv<V>(wb, a.wb + c0);
#pragma unroll
          for (int e = 0; e < V; ++e) y[i][e] = y[i][e] * ia * wa[e] + z[i][e] * ib * wb[e];
        });
      }
    }
    chunks([&](int i, int c0) {
      float s[V];
      ldv<V>(s, a.scale + c0);
#pragma unroll
      for (int e = 0; e < V; ++e) r[i][e] = a.alpha * r[i][e] + s[e] * y[i][e];
    });
    ln(a.w_post);
    if (!a.rows_idx) chunks([&](int i, int c0) { stv<V>(rr + c0, r[i]); });
  }
  if (a.w_pre) ln(a.w_pre);
  chunks([&](int i, int c0) { stv<V>((T*)a.out + (long)blockIdx.x * cols + c0, r[i]); });
}

int sum_norm(void* out, float* residual, const void* ya, long a_ld, int a_slabs, long a_stride,
             const int* mix_pos, const float* mix_w, int mix_n, const void* yb, long b_ld,
             int b_slabs, long b_stride, const float* wa, const float* wb, float alpha,
             const float* scale, const float* w_post, const float* w_pre, const long* rows_idx,
             int rows, int cols, float eps, int is_bf16, hipStream_t stream) {
  if (rows <= 0) return 0;
  if (cols <= 0 || !residual || !out || (ya && (!w_post || !scale)) || (!ya && !w_pre) ||
      (mix_pos && (!ya || !mix_w || a_slabs || yb)) || (yb && (!ya || !wa || !wb)))
    return -1;
  const SumNormArgs a{out, residual, {ya, a_ld, a_stride, a_slabs}, {yb, b_ld, b_stride, b_slabs},
                      mix_pos, mix_w, mix_n, wa, wb, alpha, scale, w_post, w_pre, rows_idx, cols, eps};
  const bool vec = cols % 8 == 0 && a_ld % 8 == 0 && b_ld % 8 == 0 &&
                   (((uintptr_t)ya | (uintptr_t)yb) & 15) == 0;
  const int nchunk = vec ? cols / 8 : cols;
  const int vpt = (nchunk + 511) / 512;
  if (vpt > (vec ? 4 : 8)) return -2;
  const int threads = nchunk >= 512 ? 512 : (nchunk + 63) / 64 * 64;
#define LMX_SN(T, V, P) sum_norm_kernel<T, V, P><<<dim3(rows), dim3(threads), 0, stream>>>(a)
#define LMX_SNT(T)                                                            \
  if (vec) {                                                                  \
    if (vpt == 1) LMX_SN(T, 8, 1); else if (vpt == 2) LMX_SN(T, 8, 2);        \
    else LMX_SN(T, 8, 4);                                                     \
  } else {                                                                    \
    if (vpt == 1) LMX_SN(T, 1, 1); else LMX_SN(T, 1, 8);                      \
  }
  if (is_bf16) { LMX_SNT(bf16_t) } else { LMX_SNT(float) }
#undef LMX_SNT
#undef LMX_SN
  return (int)hipGetLastError();
}

// Gated RMS norm of a mixer's output, in `groups` equal parts of a row, each
// divided by its own root mean square:
//   mode 0: out = norm(x) * w * sigmoid(g)      (linear attention)
//   mode 1: out = norm(x * silu(g)) * w         (state-space mixer)
//   mode 2: out = norm(x) * w * silu(g)         (retention, delta rule)
// grid (rows, groups), one workgroup per part; parts of up to 512 columns with
// a power of two of 8-column pieces: one lane group per part, grid (row blocks).
template <typename T, int V, int VPT>
__global__ void __launch_bounds__(256) gated_norm_kernel(T* out, long out_ld, const T* x, long x_ld,
                                                         const T* g, long g_ld,
                                                         const float* __restrict__ w, int part,
                                                         int mode, float eps) {
  __shared__ float scratch[16];
  const long row = blockIdx.x, off = (long)blockIdx.y * part;
  const T* xr = x + row * x_ld + off;
  const T* gr = g + row * g_ld + off;
  const int nchunk = part / V;
  float v[VPT][V], gt[VPT][V];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c >= nchunk) continue;
    ldv<V>(v[i], xr + c * V);
    ldv<V>(gt[i], gr + c * V);
#pragma unroll
    for (int e = 0; e < V; ++e) {
      const float s = sigmoid_t<T>(gt[i][e]);
      if (mode == 1) v[i][e] *= gt[i][e] * s;
      gt[i][e] = mode == 0 ? s : mode == 1 ? 1.f : gt[i][e] * s;
      ss += v[i][e] * v[i][e];
    }
  }
  ss = block_sum(ss, scratch);
  const float inv = rsqrtf(ss / (float)part + eps);
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c >= nchunk) continue;
    float wv[V];
    ldv<V>(wv, w + off + c * V);
#pragma unroll
    for (int e = 0; e < V; ++e) wv[e] *= v[i][e] * inv * gt[i][e];
    stv<V>(out + row * out_ld + off + c * V, wv);
  }
}

// lanes = part / 8 (a power of two up to 64): a part is one aligned lane group
template <typename T>
__global__ void __launch_bounds__(256) gated_norm_lanes_kernel(
    T* out, long out_ld, const T* x, long x_ld, const T* g, long g_ld,
    const float* __restrict__ w, long pieces, int per_row, int lanes, int mode, float eps) {
  const long e0 = (long)blockIdx.x * 256 + threadIdx.x;
  const bool on = e0 < pieces;
  const long it = on ? e0 : pieces - 1;         // every lane takes part in the exchange
  const long row = it / per_row;
  const int c0 = 8 * (int)(it - row * per_row);
  float v[8], gt[8], wv[8], ss = 0.f;
  ldv<8>(v, x + row * x_ld + c0);
  ldv<8>(gt, g + row * g_ld + c0);
  ldv<8>(wv, w + c0);
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    const float s = sigmoid_t<T>(gt[e]);
    if (mode == 1) v[e] *= gt[e] * s;
    wv[e] *= mode == 0 ? s : mode == 1 ? 1.f : gt[e] * s;
    ss += v[e] * v[e];
  }
  for (int o = lanes >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
  const float inv = rsqrtf(ss / (float)(8 * lanes) + eps);
#pragma unroll
  for (int e = 0; e < 8; ++e) wv[e] *= v[e] * inv;
  if (on) stv<8>(out + row * out_ld + c0, wv);
}

int gated_norm(void* out, long out_ld, const void* x, long x_ld, const void* g, long g_ld,
               const float* w, int rows, int cols, int groups, int mode, float eps,
               int is_bf16, hipStream_t stream) {
  if (rows <= 0) return 0;
  if (groups < 1 || cols % groups != 0 || mode < 0 || mode > 2) return -1;
  const int part = cols / groups;
  const bool vec = part % 8 == 0 && out_ld % 8 == 0 && x_ld % 8 == 0 && g_ld % 8 == 0 &&
                   (((uintptr_t)x | (uintptr_t)g | (uintptr_t)out) & 15) == 0;
  const int nchunk = vec ? part / 8 : part, vpt = (nchunk + 255) / 256;
  if (vpt > (vec ? 8 : 16)) return -2;
  if (vec && nchunk <= 64 && (nchunk & (nchunk - 1)) == 0) {
    const long pieces = (long)rows * (cols / 8);
    const dim3 gl((unsigned)((pieces + 255) / 256));
    if (is_bf16)
      gated_norm_lanes_kernel<bf16_t><<<gl, dim3(256), 0, stream>>>(
          (bf16_t*)out, out_ld, (const bf16_t*)x, x_ld, (const bf16_t*)g, g_ld, w, pieces, cols / 8,
          nchunk, mode, eps);
    else
      gated_norm_lanes_kernel<float><<<gl, dim3(256), 0, stream>>>(
          (float*)out, out_ld, (const float*)x, x_ld, (const float*)g, g_ld, w, pieces, cols / 8,
          nchunk, mode, eps);
    return (int)hipGetLastError();
  }
  const int threads = nchunk >= 256 ? 256 : (nchunk + 63) / 64 * 64;
  const dim3 grid(rows, groups);
#define LMX_GN(T, V, P)                                                                         \
  gated_norm_kernel<T, V, P><<<grid, dim3(threads), 0, stream>>>(                               \
      (T*)out, out_ld, (const T*)x, x_ld, (const T*)g, g_ld, w, part, mode, eps)
#define LMX_GNT(T)                                                                              \
  if (vec) {                                                                                    \
    if (vpt == 1) LMX_GN(T, 8, 1); else if (vpt == 2) LMX_GN(T, 8, 2); else LMX_GN(T, 8, 8);    \
  } else {                                                                                      \
    if (vpt == 1) LMX_GN(T, 1, 1); else LMX_GN(T, 1, 16);                                       \
  }
  if (is_bf16) { LMX_GNT(bf16_t) } else { LMX_GNT(float) }
#undef LMX_GNT
#undef LMX_GN
  return (int)hipGetLastError();
}

}  // namespace lmx
