// K18: mixture-of-experts routing.
//
//   moe_route  router logits in fp32, the top experts of every row (lowest
//              index first among equals) and the softmax over just those; then
//              `extra` further experts every row uses with weight 1.  Or by
//              scores s = sigmoid(logit): the top s + correction among the best
//              groups of neighbouring experts, in the proportions of their s; the
//              extra ones then weigh sigmoid of one more logit.  Or by s = softmax
//              over all logits, groups ranked by their largest score, weighted by s
//              itself.  The last `identity` experts return their input: they are no
//              uses (id -1), their weights are summed per row.
//              bf16 rows, up to 128 experts: 16 rows per workgroup on MFMA, the K
//              range split over the waves; otherwise one row per workgroup on the VALU.
//   moe_plan   the uses (row, expert) sorted by expert: expert row ranges, the
//              row of every sorted use and the sorted place of every use, and
//              the row tiles of the grouped products (grouped.hip).
#include "common.h"

namespace lmx {
namespace {

constexpr int MAXE = 256, MAXTOP = 32;

struct RouteBy {
  const float* correction;   // [E]: scores of all experts; null: softmax over the top logits
  int groups, keep;
  int rows;                  // router rows: E, or E + 1 with the extra experts' logit
  int softmax;               // the scores are a softmax, else sigmoids
  int identity;              // of the E
};

// One wave ranks one row's logits z[E] (LDS) and writes its uses.
__device__ __forceinline__ void moe_select(float* z, int E, int top, int extra, const RouteBy& by,
                                           int* ids, float* wts, float* own) {
  const int lane = threadIdx.x & 63;
  float v[MAXE / 64];
  float more = 1.f;          // weight of the extra experts
  if (by.correction) {
    // z becomes the scores, v the choice scores of the kept groups
    if (by.rows > E) more = 1.f / (1.f + expf(-z[E]));
    float zmax = -INFINITY, zsum = 0.f;
    if (by.softmax) {
      for (int e = lane; e < E; e += 64) zmax = fmaxf(zmax, z[e]);
      zmax = wave_max(zmax);
      for (int e = lane; e < E; e += 64) zsum += expf(z[e] - zmax);
      zsum = wave_sum(zsum);
    }
#pragma unroll
    for (int i = 0; i < MAXE / 64; ++i) {
      const int e = i * 64 + lane;
      v[i] = -INFINITY;
      if (e < E) {
        const float s = by.softmax ? expf(z[e] - zmax) / zsum : 1.f / (1.f + expf(-z[e]));
        z[e] = s;
        v[i] = s + by.correction[e];
      }
    }
    __builtin_amdgcn_wave_barrier();
    const int size = E / by.groups;
    float a = -INFINITY, b = -INFINITY;       // the two largest of lane's group
    if (lane < by.groups)
      for (int e = lane * size; e < (lane + 1) * size; ++e) {
        const float c = z[e] + by.correction[e];
        if (c > a) { b = a; a = c; } else if (c > b) { b = c; }
      }
    const float score = lane < by.groups ? a + (size > 1 && !by.softmax ? b : 0.f) : -INFINITY;
    int rank = 0;
    for (int g = 0; g < by.groups; ++g) {
      const float o = __shfl(score, g, 64);
      rank += o > score || (o == score && g < lane);
    }
    const unsigned long long kept = __ballot(lane < by.groups && rank < by.keep);
#pragma unroll
    for (int i = 0; i < MAXE / 64; ++i) {
      const int e = i * 64 + lane;
      if (e < E && !(kept >> (e / size) & 1)) v[i] = -INFINITY;
    }
  } else {
#pragma unroll
    for (int i = 0; i < MAXE / 64; ++i) v[i] = i * 64 + lane < E ? z[i * 64 + lane] : -INFINITY;
  }
  float first = 0.f, mine = 0.f, sum = 0.f;
  int id = 0;
  for (int j = 0; j < top; ++j) {
    float best = v[0];
    int at = lane;
#pragma unroll
    for (int i = 1; i < MAXE / 64; ++i)
      if (v[i] > best) { best = v[i]; at = i * 64 + lane; }
    if (best == -INFINITY) at = MAXE;         // a lane with nothing left loses every tie
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ov = __shfl_xor(best, o, 64);
      const int oa = __shfl_xor(at, o, 64);
      if (ov > best || (ov == best && oa < at)) { best = ov; at = oa; }
    }
    if (at >= E) at = E - 1;                  // NaN logits: any valid expert
#pragma unroll
    for (int i = 0; i < MAXE / 64; ++i)
      if (i * 64 + lane == at) v[i] = -INFINITY;
    if (j == 0) first = best;
    const float w = by.correction ? z[at] : expf(best - first);
    sum += w;
    if (lane == j) { mine = w; id = at; }
  }
  const int real = E - by.identity;
  const bool same = lane < top && id >= real;        // an identity expert
  if (own) {
    const float w = wave_sum(same ? mine : 0.f);
    if (lane == 0) *own = w;
  }
  if (lane < top) {
    ids[lane] = same ? -1 : id;
    wts[lane] = same ? 0.f : by.softmax ? mine : mine / (by.correction ? sum + 1e-20f : sum);
  } else if (lane < top + extra) {
    ids[lane] = real + lane - top;
    wts[lane] = more;
  }
}

// grid ceil(T / 16), block 64 NW: NW waves split the K range
template <int NT, int NW>
__global__ void __launch_bounds__(64 * NW) moe_route_mfma_kernel(
    const bf16_t* __restrict__ h, long h_ld, const bf16_t* __restrict__ w, int T, int d, int E,
    int top, int extra, RouteBy by, int* __restrict__ ids, float* __restrict__ wts,
    float* __restrict__ own) {
  __shared__ float part[NW][16][NT * 16 + 1];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c = lane & 15, q = lane >> 4;
  const int t0 = blockIdx.x * 16;
  const bf16_t* hr = h + (long)min(t0 + c, T - 1) * h_ld + 8 * q;
  const bf16_t* wr[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) wr[i] = w + (long)min(16 * i + c, by.rows - 1) * d + 8 * q;
  f32x4_t acc[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) acc[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  const bf16x8_t zero = {0, 0, 0, 0, 0, 0, 0, 0};
  const int kc = ((d + 31) / 32 + NW - 1) / NW * 32;      // whole K32 steps per wave
  const int k1 = min((wave + 1) * kc, d);
  int k0 = wave * kc;
  constexpr int U = NT <= 2 ? 8 : 4;
  for (; k0 + 32 * U <= k1; k0 += 32 * U) {
    bf16x8_t x[U], wv[U][NT];
#pragma unroll
    for (int s = 0; s < U; ++s) {
      x[s] = load_frag16B(hr + k0 + 32 * s);
#pragma unroll
      for (int i = 0; i < NT; ++i) wv[s][i] = load_frag16B(wr[i] + k0 + 32 * s);
    }
#pragma unroll
    for (int s = 0; s < U; ++s)
#pragma unroll
      for (int i = 0; i < NT; ++i) acc[i] = mfma16(wv[s][i], x[s], acc[i]);  // row = expert, column = token
  }
  for (; k0 < k1; k0 += 32) {
    const bool in = k0 + 8 * q < d;                      // d is a multiple of 8
    const bf16x8_t x = in ? load_frag16B(hr + k0) : zero;
#pragma unroll
    for (int i = 0; i < NT; ++i)
      acc[i] = mfma16(in ? load_frag16B(wr[i] + k0) : zero, x, acc[i]);
  }
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) part[wave][c][16 * i + 4 * q + r] = acc[i][r];
  __syncthreads();
  for (int e = threadIdx.x; e < 16 * NT * 16; e += 64 * NW) {
    const int t = e / (NT * 16), n = e % (NT * 16);
    float s = part[0][t][n];
#pragma unroll
    for (int v = 1; v < NW; ++v) s += part[v][t][n];
    part[0][t][n] = s;
  }
  __syncthreads();
  for (int t = wave; t < 16; t += NW)
    if (t0 + t < T)
      moe_select(part[0][t], E, top, extra, by, ids + (long)(t0 + t) * (top + extra),
                 wts + (long)(t0 + t) * (top + extra), own ? own + t0 + t : nullptr);
}

// grid T, block 256
template <typename T_>
__global__ void __launch_bounds__(256) moe_route_any_kernel(const T_* __restrict__ h, long h_ld,
                                                            const T_* __restrict__ w, int d, int E,
                                                            int top, int extra, RouteBy by,
                                                            int* __restrict__ ids,
                                                            float* __restrict__ wts,
                                                            float* __restrict__ own) {
  __shared__ float z[MAXE];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const long t = blockIdx.x;
  for (int e = wave; e < by.rows; e += 4) {
    float s = 0.f;
    for (int k = lane; k < d; k += 64) s += ld1(h + t * h_ld + k) * ld1(w + (long)e * d + k);
    s = wave_sum(s);
    if (lane == 0) z[e] = s;
  }
  __syncthreads();
  if (wave == 0)
    moe_select(z, E, top, extra, by, ids + t * (top + extra), wts + t * (top + extra),
               own ? own + t : nullptr);
}

constexpr int CHUNK = 1024;      // uses per block of the sort (ops MOE_CHUNK)
constexpr int SMALL = 8192;      // uses one workgroup sorts alone

struct PlanArgs {
  const int* ids;
  int n, J, groups, bm, mtiles, blocks;
  int *hist, *off, *src, *pos;
  int* tiles;              // [mtiles][2], then the number of used ones
};

// expert ranges and tiles from the counts cnt[groups] (LDS); beg[] gets the
// first places.  Whole workgroup.
__device__ __forceinline__ void plan_ranges(const PlanArgs& p, const int* cnt, int* beg, int* tbeg) {
  if (threadIdx.x == 0) {
    int a = 0, t = 0;
    for (int g = 0; g < p.groups; ++g) {
      beg[g] = a;
      tbeg[g] = t;
      a += cnt[g];
      t += (cnt[g] + p.bm - 1) / p.bm;
    }
    beg[p.groups] = a;
    tbeg[p.groups] = t;
  }
  __syncthreads();
  for (int g = threadIdx.x; g <= p.groups; g += blockDim.x) p.off[g] = beg[g];
  if (threadIdx.x == 0) p.tiles[2 * p.mtiles] = tbeg[p.groups];
  for (int t = threadIdx.x; t < p.mtiles; t += blockDim.x) {
    int g = -1, r = 0;
    if (t < tbeg[p.groups]) {
      int lo = 0, hi = p.groups - 1;           // last group with tbeg <= t
      while (lo < hi) {
        const int mid = (lo + hi + 1) >> 1;
        if (tbeg[mid] <= t) lo = mid; else hi = mid - 1;
      }
      g = lo;
      r = beg[g] + (t - tbeg[g]) * p.bm;
    }
    p.tiles[2 * t] = g;
    p.tiles[2 * t + 1] = r;
  }
}

__device__ __forceinline__ void place_use(const PlanArgs& p, int i, int* next) {
  const int g = p.ids[i];
  const int at = g < 0 ? -1 : atomicAdd(&next[g], 1);
  if (at >= 0) p.src[at] = i / p.J;
  p.pos[i] = at;
}

__global__ void __launch_bounds__(1024) moe_plan_small_kernel(PlanArgs p) {
  __shared__ int cnt[MAXE], beg[MAXE + 1], tbeg[MAXE + 1];
  for (int g = threadIdx.x; g < p.groups; g += blockDim.x) cnt[g] = 0;
  __syncthreads();
  for (int i = threadIdx.x; i < p.n; i += blockDim.x)
    if (p.ids[i] >= 0) atomicAdd(&cnt[p.ids[i]], 1);
  __syncthreads();
  plan_ranges(p, cnt, beg, tbeg);
  __syncthreads();
  for (int i = threadIdx.x; i < p.n; i += blockDim.x) place_use(p, i, beg);
}

__global__ void __launch_bounds__(256) moe_hist_kernel(PlanArgs p) {
  __shared__ int cnt[MAXE];
  for (int g = threadIdx.x; g < p.groups; g += 256) cnt[g] = 0;
  __syncthreads();
  const int i1 = min(p.n, (int)(blockIdx.x + 1) * CHUNK);
  for (int i = blockIdx.x * CHUNK + threadIdx.x; i < i1; i += 256)
    if (p.ids[i] >= 0) atomicAdd(&cnt[p.ids[i]], 1);
  __syncthreads();
  for (int g = threadIdx.x; g < p.groups; g += 256) p.hist[blockIdx.x * p.groups + g] = cnt[g];
}

// one workgroup: hist[b][g] becomes the place of block b's first use of g
__global__ void __launch_bounds__(1024) moe_scan_kernel(PlanArgs p) {
  __shared__ int cnt[MAXE], beg[MAXE + 1], tbeg[MAXE + 1];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  for (int g = wave; g < p.groups; g += 16) {
    int run = 0;
    for (int b0 = 0; b0 < p.blocks; b0 += 64) {
      const int b = b0 + lane, v = b < p.blocks ? p.hist[b * p.groups + g] : 0;
      int s = v;
      for (int o = 1; o < 64; o <<= 1) {
        const int x = __shfl_up(s, o, 64);
        if (lane >= o) s += x;
      }
      if (b < p.blocks) p.hist[b * p.groups + g] = run + s - v;
      run += __shfl(s, 63, 64);
    }
    if (lane == 0) cnt[g] = run;
  }
  __syncthreads();
  plan_ranges(p, cnt, beg, tbeg);
}

__global__ void __launch_bounds__(256) moe_scatter_kernel(PlanArgs p) {
  __shared__ int next[MAXE];
  for (int g = threadIdx.x; g < p.groups; g += 256)
    next[g] = p.off[g] + p.hist[blockIdx.x * p.groups + g];
  __syncthreads();
  const int i1 = min(p.n, (int)(blockIdx.x + 1) * CHUNK);
  for (int i = blockIdx.x * CHUNK + threadIdx.x; i < i1; i += 256) place_use(p, i, next);
}

}  // namespace

int moe_route(const void* h, long h_ld, const void* w, int T, int d, int E, int rows, int top,
              int extra, const float* correction, int groups, int keep, int softmax, int identity,
              int* ids, float* wts, float* own, int is_bf16, hipStream_t stream) {
  if (T <= 0) return 0;
  if (rows < E || rows > E + 1 || rows > MAXE || (rows > E && !correction) ||
      (correction && (groups < 1 || groups > 64 || E % groups || keep < 1 || keep > groups ||
                      keep * (E / groups) < top)))
    return -1;
  if ((softmax || identity) && (!correction || rows > E)) return -1;
  if (identity < 0 || identity >= E || (identity > 0) != (own != nullptr)) return -1;
  const RouteBy by{correction, groups, keep, rows, softmax, identity};
  if (E < 1 || E > MAXE || top < 1 || top > E || extra < 0 || top + extra > MAXTOP || d < 1)
    return -1;
  if (is_bf16 && rows <= 128 && d % 8 == 0 && h_ld % 8 == 0 && !(((uintptr_t)h | (uintptr_t)w) & 15)) {
    const int nt = (rows + 15) / 16;
#define LMX_RT(NT, NW)                                                                       \
  moe_route_mfma_kernel<NT, NW><<<dim3((T + 15) / 16), dim3(64 * NW), 0, stream>>>(          \
      (const bf16_t*)h, h_ld, (const bf16_t*)w, T, d, E, top, extra, by, ids, wts, own)
    if (nt == 1) LMX_RT(1, 16); else if (nt == 2) LMX_RT(2, 16); else if (nt <= 4) LMX_RT(4, 8);
    else LMX_RT(8, 4);
#undef LMX_RT
  } else if (is_bf16) {
    moe_route_any_kernel<bf16_t><<<dim3(T), dim3(256), 0, stream>>>(
        (const bf16_t*)h, h_ld, (const bf16_t*)w, d, E, top, extra, by, ids, wts, own);
  } else {
    moe_route_any_kernel<float><<<dim3(T), dim3(256), 0, stream>>>(
        (const float*)h, h_ld, (const float*)w, d, E, top, extra, by, ids, wts, own);
  }
  return (int)hipGetLastError();
}

// every id is in -1..groups - 1 (moe_route's; -1: no use)
int moe_plan(const int* ids, int n, int J, int groups, int bm, int mtiles, int* hist, int* off,
             int* src, int* pos, int* tiles, hipStream_t stream) {
  if (n <= 0) return 0;
  if (groups < 1 || groups > MAXE || J < 1 || bm < 1 || mtiles < 1) return -1;
  const PlanArgs p{ids, n, J, groups, bm, mtiles, (n + CHUNK - 1) / CHUNK,
                   hist, off, src, pos, tiles};
  if (n <= SMALL) {
    moe_plan_small_kernel<<<dim3(1), dim3(1024), 0, stream>>>(p);
  } else {
    moe_hist_kernel<<<dim3(p.blocks), dim3(256), 0, stream>>>(p);
    moe_scan_kernel<<<dim3(1), dim3(1024), 0, stream>>>(p);
    moe_scatter_kernel<<<dim3(p.blocks), dim3(256), 0, stream>>>(p);
  }
  return (int)hipGetLastError();
}

}  // namespace lmx
