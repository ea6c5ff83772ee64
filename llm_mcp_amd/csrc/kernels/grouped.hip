// K17: grouped products C[rows of g] = A[rows of g] . W[g]^T.
//
// Two forms of "rows of g":
//   heads    every row belongs to every group; group g reads A's columns from
//            g * a_gs and writes C's from g * c_gs (per-head maps of latent
//            attention)
//   experts  rows sorted by group (moe_plan): a tile list names each tile's
//            group and first row, src (optional) the A row of a sorted row
// Epilogues: none; a clamped GLU over 16-column gate / up pairs
//   g = min(gate, L), u = clamp(up, -L, L), g sigmoid(slope g) (u + shift)
//   (SiLU-GLU: no clamp, slope 1, shift 0);
// or a multiplication with sigmoid(gate rows).
//
// bf16 weights come packed in MFMA fragment order,
//   [g][N / 16][K / 32][lane: 16 (k / 8) + n][8 of k],
// so a wave's fragment load is one contiguous KB, from HBM to registers
// (small-M kernel) or to LDS by DMA without a swizzle (large-M kernel).  MFMA
// operands are swapped (D = W . A^T): a lane's 4 accumulators are 4
// consecutive output columns of one row.
//
//   grouped_small   BM x 64 tiles, BM = 16 / 32 / 64: decode batches, bound by the
//                   weight stream; A in LDS, one 16-column tile per wave
//   grouped_large   128 x 128 tiles of 64-deep K steps, double-buffered
//                   LDS-DMA, 4 waves of 64 x 64
//   grouped_f32     fp32 rows and weights [g][N][K], 32 x 32 tiles
#include "common.h"

namespace lmx {
namespace {

struct GroupArgs {
  const void* a;
  long lda, a_gs;
  const void* w;
  void* c;
  long ldc, c_gs;
  int N, K, M;            // M: rows of every group (heads), sorted rows (experts)
  const int* tiles;       // experts: [mt][2] (group or -1, first row); null: heads
  const int* off;         // experts: [groups + 1] first rows
  const int* src;         // experts: A row of a sorted row; null: the row itself
  const float* limit;     // GLU clamp per group; null: no GLU
  float slope, shift;
  const void* gate;       // sigmoid gate rows (heads); null: none
  long gate_ld;
};

// tile -> group, first row, one past the last row of this tile's group
__device__ __forceinline__ bool group_tile(const GroupArgs& p, int mt, int gz, int bm, int& g,
                                           int& r0, int& r1) {
  if (p.tiles) {
    g = p.tiles[2 * mt];
    if (g < 0) return false;
    r0 = p.tiles[2 * mt + 1];
    r1 = p.off[g + 1];
  } else {
    g = gz;
    r0 = mt * bm;
    r1 = p.M;
  }
  return r0 < r1;
}

template <typename T>
__device__ __forceinline__ float clamped_glu(const GroupArgs& p, float g, float u, float lim) {
  g = fminf(g, lim);
  u = fminf(fmaxf(u, -lim), lim);
  return g * sigmoid_t<T>(p.slope * g) * (u + p.shift);
}

// 4 consecutive columns n.. of row `row`
__device__ __forceinline__ void group_store(const GroupArgs& p, int g, long row, int n, f32x4_t v) {
  if (p.gate) {
    const bf16x4_t gt = *reinterpret_cast<const bf16x4_t*>(
        (const bf16_t*)p.gate + row * p.gate_ld + (long)g * p.c_gs + n);
#pragma unroll
    for (int r = 0; r < 4; ++r) v[r] /= 1.f + __expf(-bf2f((uint16_t)gt[r]));
  }
  bf16x4_t o;
#pragma unroll
  for (int r = 0; r < 4; ++r) o[r] = (short)f2bf(v[r]);
  *reinterpret_cast<bf16x4_t*>((bf16_t*)p.c + row * p.ldc + (long)g * p.c_gs + n) = o;
}

__device__ __forceinline__ f32x4_t glu4(const GroupArgs& p, f32x4_t g, f32x4_t u, float lim) {
  f32x4_t o;
#pragma unroll
  for (int r = 0; r < 4; ++r) o[r] = clamped_glu<bf16_t>(p, g[r], u[r], lim);
  return o;
}

// ------------------------------------------------------------- decode rows ----
// grid (N / 64, row tiles, groups | 1), block 256.  A is staged in chunks of
// SK columns: image [BM][SK], 16-B chunks XOR-swizzled by the row.
constexpr int SK = 256;

template <int BM>
__global__ void __launch_bounds__(256) grouped_small_kernel(GroupArgs p) {
  __shared__ __attribute__((aligned(16))) bf16_t sa[2][BM * SK];
  int g, r0, r1;
  if (!group_tile(p, blockIdx.y, blockIdx.z, BM, g, r0, r1)) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, q = lane >> 4;
  const int nt = blockIdx.x * 4 + wave;                 // 16-column tile
  const bool on = nt * 16 < p.N;
  const int K32 = p.K / 32;
  const bf16_t* wp = (const bf16_t*)p.w + ((long)g * (p.N / 16) + (on ? nt : 0)) * K32 * 512 +
                     lane * 8;
  constexpr int PER = BM * SK / 8 / 256;                // A pieces of 16 B per thread and chunk
  // source rows of this thread's pieces (fixed over the chunks)
  const bf16_t* ar[PER];
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int row = min(r0 + (i * 256 + tid) / (SK / 8), r1 - 1);
    ar[i] = (const bf16_t*)p.a + (long)(p.src ? p.src[row] : row) * p.lda + (long)g * p.a_gs;
  }
  auto stage = [&](int k0, int buf) {
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int e = i * 256 + tid, row = e / (SK / 8), ch = (e % (SK / 8)) ^ (row & 15);
      const int k = min(k0 + 8 * ch, p.K - 8);          // past K: any valid columns, unused
      lds_dma16(ar[i] + k, &sa[buf][(i * 256 + wave * 64) * 8]);
    }
  };
  constexpr int MT = BM / 16, KS = SK / 32;
  f32x4_t acc[MT];
#pragma unroll
  for (int i = 0; i < MT; ++i) acc[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  bf16x8_t wf[KS], wn[KS];
  auto load_w = [&](bf16x8_t (&f)[KS], int k0) {
#pragma unroll
    for (int s = 0; s < KS; ++s)
      f[s] = __builtin_nontemporal_load(
          reinterpret_cast<const bf16x8_t*>(wp + (long)min(k0 / 32 + s, K32 - 1) * 512));
  };
  stage(0, 0);
  load_w(wf, 0);
  int buf = 0;
  for (int k0 = 0; k0 < p.K; k0 += SK) {
    dma_barrier();                    // this chunk landed; the other buffer is free
    // ... and so did its weights: the compiler must not wait for them again,
    // behind the next chunk's loads
#pragma unroll
    for (int s = 0; s < KS; ++s) asm volatile("" : "+v"(wf[s]));
    if (k0 + SK < p.K) {
      stage(k0 + SK, buf ^ 1);
      load_w(wn, k0 + SK);
    }
    auto step = [&](int s) {
#pragma unroll
      for (int i = 0; i < MT; ++i) {
        const int row = 16 * i + c;
        acc[i] = mfma16(wf[s], load_frag16B(&sa[buf][row * SK + 8 * ((4 * s + q) ^ (row & 15))]),
                        acc[i]);
      }
    };
    if (k0 + SK <= p.K) {
#pragma unroll
      for (int s = 0; s < KS; ++s) step(s);
    } else {
#pragma unroll
      for (int s = 0; s < KS; ++s)
        if (k0 + 32 * s < p.K) step(s);
    }
#pragma unroll
    for (int s = 0; s < KS; ++s) wf[s] = wn[s];
    buf ^= 1;
  }
  if (p.limit) {
    // gate and up tiles sit in neighbouring waves: exchange through LDS
    __syncthreads();
    f32x4_t* ex = reinterpret_cast<f32x4_t*>(&sa[0][0]);
    if (wave & 1)
#pragma unroll
      for (int i = 0; i < MT; ++i) ex[((wave >> 1) * MT + i) * 64 + lane] = acc[i];
    __syncthreads();
    if ((wave & 1) || !on) return;
    const float lim = p.limit[g];
#pragma unroll
    for (int i = 0; i < MT; ++i) {
      const int row = r0 + 16 * i + c;
      const f32x4_t o = glu4(p, acc[i], ex[((wave >> 1) * MT + i) * 64 + lane], lim);
      if (row < r1) group_store(p, g, row, nt / 2 * 16 + 4 * q, o);
    }
    return;
  }
  if (!on) return;
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    const int row = r0 + 16 * i + c;
    if (row < r1) group_store(p, g, row, nt * 16 + 4 * q, acc[i]);
  }
}

// ------------------------------------------------------------- prompt rows ----
// grid (N tiles x row tiles, groups | 1), block 256 = 2 x 2 waves of 64 x 64.
constexpr int LBM = 128, LBN = 128, LBK = 64;

__global__ void __launch_bounds__(256, 2) grouped_large_kernel(GroupArgs p, int mtiles) {
  __shared__ __attribute__((aligned(16))) bf16_t sa[2][LBM * LBK];
  __shared__ __attribute__((aligned(16))) bf16_t sw[2][LBN * LBK];
  const int ntiles = (p.N + LBN - 1) / LBN;
  // one XCD's consecutive workgroups: 8 row tiles under one column tile after
  // the other, so their A rows and the column's weights stay in its L2
  const int lin = xcd_remap(blockIdx.x, gridDim.x);
  const int per = 8 * ntiles, gi = lin / per, rem = lin % per;
  const int gs = min(8, mtiles - gi * 8);
  const int mt = gi * 8 + rem % gs, ntl = rem / gs;
  int g, r0, r1;
  if (!group_tile(p, mt, blockIdx.y, LBM, g, r0, r1)) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, q = lane >> 4;
  const int wm = wave & 1, wn = wave >> 1;
  const int K32 = p.K / 32, n16 = p.N / 16;
  // A: 128 rows x 8 chunks; 4 pieces per thread
  const bf16_t* ar[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int e = i * 256 + tid, rr = e >> 3, ch = (e & 7) ^ (rr & 7);
    const int row = min(r0 + rr, r1 - 1);
    ar[i] = (const bf16_t*)p.a + (long)(p.src ? p.src[row] : row) * p.lda + (long)g * p.a_gs +
            8 * ch;
  }
  // W: 8 column tiles x 2 k32 blocks of 1 KB; each wave copies 4 of them
  const bf16_t* wr[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int blk = i * 4 + wave, t = min(ntl * 8 + (blk >> 1), n16 - 1);
    wr[i] = (const bf16_t*)p.w + (((long)g * n16 + t) * K32 + (blk & 1)) * 512 + lane * 8;
  }
  auto stage = [&](int ks, int buf) {
#pragma unroll
    for (int i = 0; i < 4; ++i) lds_dma16(ar[i] + ks * LBK, &sa[buf][(i * 256 + wave * 64) * 8]);
#pragma unroll
    for (int i = 0; i < 4; ++i)
      lds_dma16(wr[i] + (long)ks * 1024, &sw[buf][(i * 4 + wave) * 512]);
  };
  f32x4_t acc[4][4];                   // [row tile][column tile]
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  const int nk = p.K / LBK;
  stage(0, 0);
  for (int ks = 0; ks < nk; ++ks) {
    const int buf = ks & 1;
    dma_barrier();                     // step ks landed; every wave is done with the other buffer
    if (ks + 1 < nk) stage(ks + 1, buf ^ 1);
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      bf16x8_t af[4], wf[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int row = wm * 64 + 16 * i + c;
        af[i] = load_frag16B(&sa[buf][row * LBK + 8 * ((4 * kk + q) ^ (row & 7))]);
      }
#pragma unroll
      for (int j = 0; j < 4; ++j)
        wf[j] = load_frag16B(&sw[buf][((wn * 4 + j) * 2 + kk) * 512 + lane * 8]);
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = mfma16(wf[j], af[i], acc[i][j]);
    }
  }
  const float lim = p.limit ? p.limit[g] : 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int row = r0 + wm * 64 + 16 * i + c;
    if (row >= r1) continue;
    if (p.limit) {
#pragma unroll
      for (int j = 0; j < 4; j += 2) {
        const int t = ntl * 8 + wn * 4 + j;
        if (t < n16) group_store(p, g, row, t / 2 * 16 + 4 * q, glu4(p, acc[i][j], acc[i][j + 1], lim));
      }
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int t = ntl * 8 + wn * 4 + j;
        if (t < n16) group_store(p, g, row, t * 16 + 4 * q, acc[i][j]);
      }
    }
  }
}

// --------------------------------------------------------------------- fp32 ----
// grid (ceil(N / 32), row tiles of 32, groups | 1), block 256
__global__ void __launch_bounds__(256) grouped_f32_kernel(GroupArgs p) {
  __shared__ float sa[32][33], sw[32][33];
  int g, r0, r1;
  if (!group_tile(p, blockIdx.y, blockIdx.z, 32, g, r0, r1)) return;
  const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4;
  const int n0 = blockIdx.x * 32;
  float acc[2][2] = {{0.f, 0.f}, {0.f, 0.f}};
  for (int k0 = 0; k0 < p.K; k0 += 32) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int e = i * 256 + tid, r = e >> 5, k = e & 31;
      const int row = r0 + r, n = n0 + r;
      sa[r][k] = row < r1 && k0 + k < p.K
                     ? ((const float*)p.a)[(long)(p.src ? p.src[row] : row) * p.lda +
                                           (long)g * p.a_gs + k0 + k] : 0.f;
      sw[r][k] = n < p.N && k0 + k < p.K
                     ? ((const float*)p.w)[((long)g * p.N + n) * p.K + k0 + k] : 0.f;
    }
    __syncthreads();
#pragma unroll 8
    for (int k = 0; k < 32; ++k)
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i][j] += sa[ty + 16 * i][k] * sw[tx + 16 * j][k];
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int row = r0 + ty + 16 * i;
    if (row >= r1) continue;
    float* cr = (float*)p.c + row * p.ldc + (long)g * p.c_gs;
    if (p.limit) {                     // columns n0.. are 16 gate, 16 up
      if (n0 + 16 + tx < p.N) cr[n0 / 2 + tx] = clamped_glu<float>(p, acc[i][0], acc[i][1], p.limit[g]);
      continue;
    }
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int n = n0 + tx + 16 * j;
      if (n >= p.N) continue;
      float v = acc[i][j];
      if (p.gate) v *= sigmoid_t<float>(((const float*)p.gate)[row * p.gate_ld + (long)g * p.c_gs + n]);
      cr[n] = v;
    }
  }
}

}  // namespace

// bm: rows per tile (32 fp32; 16 / 32 / 64 / 128 bf16); mtiles: row tiles (experts:
// the tile list's length)
int grouped(const void* a, long lda, long a_gs, const void* w, void* c, long ldc, long c_gs,
            int groups, int N, int K, int M, const int* tiles, int mtiles, const int* off,
            const int* src, const float* limit, float slope, float shift, const void* gate,
            long gate_ld, int bm, int is_bf16, hipStream_t stream) {
  if (M <= 0 || mtiles <= 0) return 0;
  if (groups < 1 || N < 1 || K < 1 || (tiles && (!off || gate)) || (limit && N % 32)) return -1;
  const GroupArgs p{a, lda, a_gs, w, c, ldc, c_gs, N, K, M, tiles, off, src, limit, slope, shift,
                    gate, gate_ld};
  const int gz = tiles ? 1 : groups;
  if (!is_bf16) {
    if (bm != 32) return -2;
    grouped_f32_kernel<<<dim3((N + 31) / 32, mtiles, gz), dim3(256), 0, stream>>>(p);
    return (int)hipGetLastError();
  }
  if (N % 16 || K % 64 || lda % 8 || a_gs % 8 || ldc % 4 || c_gs % 4 || gate_ld % 4 ||
      ((uintptr_t)a & 15) || ((uintptr_t)w & 15) || ((uintptr_t)c & 7) || ((uintptr_t)gate & 7))
    return -3;
  if (bm == 16)
    grouped_small_kernel<16><<<dim3((N + 63) / 64, mtiles, gz), dim3(256), 0, stream>>>(p);
  else if (bm == 32)
    grouped_small_kernel<32><<<dim3((N + 63) / 64, mtiles, gz), dim3(256), 0, stream>>>(p);
  else if (bm == 64)
    grouped_small_kernel<64><<<dim3((N + 63) / 64, mtiles, gz), dim3(256), 0, stream>>>(p);
  else if (bm == LBM)
    grouped_large_kernel<<<dim3((N + LBN - 1) / LBN * mtiles, gz), dim3(256), 0, stream>>>(p, mtiles);
  else
    return -4;
  return (int)hipGetLastError();
}

}  // namespace lmx
