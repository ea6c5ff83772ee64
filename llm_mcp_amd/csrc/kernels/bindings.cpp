// pybind11 entry points of the HIP kernel library (_lmx_kernels).
//
// The Python side (llm_mcp_amd/ops/kernels.py) validates shapes, dtypes,
// contiguity and device placement of torch tensors on the host and passes raw
// device pointers plus the current HIP stream; nothing here allocates or
// synchronises, so every launch is hipGraph-capturable.
#include <hip/hip_runtime.h>
#include <pybind11/pybind11.h>
#include <pybind11/stl.h>
#include <string>
#include <vector>
#include <stdexcept>
#include <string>

#include "delta.h"

namespace lmx {
int rmsnorm(void*, void*, const void*, const void*, int, int, long, long, float, hipStream_t);
int layernorm(void*, const void*, const void*, const void*, const void*, int, int, float,
              hipStream_t);
int rope_cache(void*, long, const int*, const float*, int, int, int, int, const int*, void*, void*,
               int, int, int, const void*, const void*, float, int, hipStream_t);
int kv_write(const void*, const void*, long, const int*, int, int, int, void*, void*, int,
             hipStream_t);
void set_decode_mode(int);
void set_slab_norm_threads(int);
void set_prefill_rescale_thr(float);
void set_prefill_stages(int);
void set_prefill_xcd(int);
int paged_decode(const void*, long, const void*, const void*, const int*, int, const int*,
                 const int*, void*,
                 long, float*, float*, int, int, int, int, int, float, int, int, const int*,
                 const float*, const int*, const void*, long, int, int, float, hipStream_t);
int paged_prefill(const void*, long, const void*, const void*, const int*, int, const int*,
                  const int*, const int*, int, void*, long, int, int, int, int, float, int, int,
                  const int*, const float*, const void*, long, int, int, float, hipStream_t);
int attention_any(const void*, long, const void*, const void*, const int*, int, const int*, int,
                  const int*, int, void*, long, const void*, long, int, int, int, int, float, int,
                  float, int, hipStream_t);
int sandwich_norm(void*, float*, const void*, long, int, long, const int*, const float*, int,
                  const float*, const float*, const int*, const void*, float, const float*, const float*, const long*, int, int,
                  float, int, hipStream_t);
int sum_norm(void*, float*, const void*, long, int, long, const int*, const float*, int,
             const void*, long, int, long, const float*, const float*, float, const float*,
             const float*, const float*, const long*, int, int, float, int, hipStream_t);
int soft_cap(void*, long, float, float, int, hipStream_t);
int rotate_rows(void*, long, void*, long, const float*, int, int, int, int, int, float,
                hipStream_t);
int norm_rope_cache(const void*, long, const float*, const float*, const float*, int, const int*,
                    const int*, int, void*, void*, void*, int, int, int, int, int, float, int,
                    hipStream_t);
int delta_recurrent(const DeltaArgs&, int, int, hipStream_t);
int delta_chunks(const DeltaArgs&, int, int, const int*, int, const int*, void*, float*,
                 hipStream_t);
int gelu(void*, long, int, hipStream_t);
int grouped(const void*, long, long, const void*, void*, long, long, int, int, int, int, const int*,
            int, const int*, const int*, const float*, float, float, const void*, long, int, int,
            hipStream_t);
int pgemm_grouped(void*, const void*, const void*, int, int, int, long, long, int, const int*, int,
                  const int*, const int*, const float*, float, float, hipStream_t);
int moe_route(const void*, long, const void*, int, int, int, int, int, int, const float*, int, int,
              int, int, int*, float*, float*, int, hipStream_t);
int bias_relu2(void*, const float*, long, int, int, hipStream_t);
int qkv_norm_rope_cache(const void*, long, const float*, const float*, const float*, const float*, int,
                        const int*, const int*, int, void*, void*, void*, int, int, int, int, int, int,
                        float, int, hipStream_t);
int talk_prefill(const void*, const void*, const void*, const void*, const float*, float, int, int, int,
                 int, const int*, int, const int*, const int*, const int*, int, const void*, long,
                 void*, long, hipStream_t);
int talk_decode(const void*, const void*, const void*, const void*, const float*, float, int, int, int,
                int, const int*, int, const int*, int, const void*, long, void*, long, float*, float*,
                int, int, hipStream_t);
int talk_any(const void*, const void*, const void*, const int*, int, const int*, int, const int*, int,
             const void*, const float*, void*, long, const void*, long, float, int, int, int, int, int,
             hipStream_t);
int memory_scan(const void*, long, const void*, long, const void*, long, const void*, const void*, long,
                const float*, float, void*, long, float*, float*, float*, const int*, const int*,
                const int*, int, int, int, int, int, int, const int*, int, const int*, int, float*,
                float*, hipStream_t);
int moe_plan(const int*, int, int, int, int, int, int*, int*, int*, int*, int*, hipStream_t);
int rglru_chunks(const void*, const void*, long, const float*, const float*, const float*, void*,
                 float*, const int*, const int*, const int*, int, int, const void*, int, const int*,
                 int, const int*, float*, hipStream_t);
int rglru_rows(const void*, const void*, long, const float*, const float*, const float*, void*,
               float*, const int*, const int*, const int*, int, int, const void*, int, hipStream_t);
int rglru_scan(const void*, const void*, long, const float*, const float*, const float*, void*,
               float*, const int*, const int*, const int*, int, int, const float*, int, int,
               hipStream_t);
int rope_angles(const int*, const double*, int, int, float, float*, hipStream_t);
int latent_prep(const void*, long, int, int, int, const float*, int, int, const float*,
                const float*, int, const int*, void*, int, int, void*, float, int, hipStream_t);
int latent_rotate(const void*, long, int, const float*, int, int, int, int, void*, long, int, int,
                  hipStream_t);
int latent_any(const void*, const void*, const int*, int, const int*, int, const int*, int, void*,
               int, int, int, float, int, int, hipStream_t);
int latent_gather(const void*, const int*, int, const int*, int, int, int, void*, hipStream_t);
int latent_prefill(const void*, long, const void*, const void*, const float*, const int*,
                   const int*, int, const int*, const int*, const void*, long, void*, long, int, int,
                   int, int, int, int, float, int, hipStream_t);
int latent_rows(const void*, const void*, const int*, int, const int*, int, const int*, int, int,
                void*, float*, float*, int, int, int, float, int, int, int, hipStream_t);
int gated_norm(void*, long, const void*, long, const void*, long, const float*, int, int, int, int,
               float, int, hipStream_t);
int short_conv(const void*, long, const float*, const float*, const float*, void*, const int*, int,
               int, const int*, const int*, const int*, int, int, void*, long, int, int, hipStream_t);
int conv_qkv_cache(const void*, long, const float*, const float*, void*, const int*, int, int, const int*,
                   const int*, const int*, int, void*, long, void*, void*, const int*, const int*,
                   int, int, int, int, int, float, float, float, int, hipStream_t);
int linear_scan(const void*, long, const void*, long, const void*, long, const void*, long,
                const float*, const float*, const float*, const float*, const float*, void*, long,
                float*, const int*, const int*, const int*, int, int, int, int, int, int,
                const float*, int, float, int, int, const int*, int, const int*, int, float*,
                float*, hipStream_t);
int sample(const void*, int, long, int, int, const float*, const int*, const float*,
           const uint64_t*, const int*, int*, float*, int, hipStream_t);
int glu(void*, const void*, long, int, int, int, int, hipStream_t);
int apply_penalties(void*, int, long, int, int, const int*, const int*, const float*, const int*,
                    int, int, hipStream_t);
int race_sample_phase(int, int, int, const void*, int, long, int, int, int, int, const float*,
                      const int*, const float*, const uint64_t*, const int*, const float*, int,
                      float*, float*, int*, float*, hipStream_t);
int embed_gather(void*, const void*, const int*, int, int, int, int, hipStream_t);
int ids_from_prev(int*, const int*, const int*, int, hipStream_t);
int mean_pool_l2(float*, float*, const void*, const int*, int, int, int, int, int, hipStream_t);
int bias_act(void*, const void*, long, int, int, hipStream_t);
int gemm_splitk(void*, const void*, const void*, float*, int*, int, int, int, long, long, long,
                int, hipStream_t);
int gemm_nt(void*, const void*, const void*, const void*, const void*, int, int, int, long, long,
            long, int, hipStream_t);
int dgemm(void*, const void*, const void*, float*, unsigned*, int, int, int, int, long, long, long,
          int, int, int, hipStream_t);
int dgemm_num_configs();
int rsgemm(void*, const void*, const void*, float*, unsigned*, int, int, int, int, long, long, long,
           int, int, int, hipStream_t);
int rsgemm_pack(void*, const void*, int, int, long, hipStream_t);
int rmsnorm_slabs(void*, void*, const float*, int, long, const void*, int, int, long, float,
                  hipStream_t);
int dgemm_config(int, int*, int*);
int dgemm_sk_pieces(int, int, int, int, int);
int pgemm(void*, const void*, const void*, const void*, int, int, int, long, long, long, int, int,
          int, int, float*, hipStream_t);
int row_scale(float*, const float*, int, const void*, long, int, int, float, hipStream_t);
int pgemm_sk(void*, const void*, const void*, void*, void*, int, int, int, int, long, long, long,
             int, int, int, hipStream_t);
long ar_region_bytes(long);
int ar_alloc(void**, long);
int ar_free(void*);
int ar_ipc_handle(void*, void*);
int ar_ipc_open(void**, const void*);
int ar_ipc_close(void*);
int ar_ipc_handle_size();
int ar_error(void*, int);
int ar_error_async(void*, void*, hipStream_t);
int allreduce_norm(void*, void*, const void*, const void*, int, int, float, int, int,
                   const unsigned long long*, long, int, int, int, int, hipStream_t);
int allreduce(void*, const void*, long, int, int, const unsigned long long*, long, int, int, int,
              hipStream_t);
}  // namespace lmx

namespace py = pybind11;
typedef unsigned long long uptr;

template <typename T>
static T* P(uptr p) { return reinterpret_cast<T*>(p); }
static hipStream_t S(uptr s) { return reinterpret_cast<hipStream_t>(s); }

static void check(int rc, const char* what) {
  if (rc != 0) {
    const char* es = rc > 0 ? hipGetErrorString((hipError_t)rc) : "invalid arguments";
    throw std::runtime_error(std::string("lmx kernel ") + what + " failed (" + std::to_string(rc) +
                             "): " + es);
  }
}

PYBIND11_MODULE(_lmx_kernels, m) {
  m.doc() = "llm_mcp_amd gfx950 HIP kernels";
  m.def("rmsnorm", [](uptr out, uptr residual, uptr x, uptr w, int rows, int cols, long in_stride,
                      long out_stride, float eps, uptr stream) {
    check(lmx::rmsnorm(P<void>(out), P<void>(residual), P<void>(x), P<void>(w), rows, cols,
                       in_stride, out_stride, eps, S(stream)),
          "rmsnorm");
  });
  m.def("layernorm", [](uptr out, uptr x, uptr residual, uptr w, uptr b, int rows, int cols,
                        float eps, uptr stream) {
    check(lmx::layernorm(P<void>(out), P<void>(x), P<void>(residual), P<void>(w), P<void>(b), rows,
                         cols, eps, S(stream)),
          "layernorm");
  });
  m.def("rope_cache", [](uptr qkv, long qkv_stride, uptr positions, uptr cos_sin, int T, int Hq,
                         int Hkv, int D, uptr slots, uptr kc, uptr vc, int BS, int rot_k,
                         int tile_from, uptr q_norm, uptr k_norm, float eps, int skip_q,
                         uptr stream) {
    check(lmx::rope_cache(P<void>(qkv), qkv_stride, P<int>(positions), P<float>(cos_sin), T, Hq, Hkv,
                          D, P<int>(slots), P<void>(kc), P<void>(vc), BS, rot_k, tile_from,
                          P<void>(q_norm), P<void>(k_norm), eps, skip_q, S(stream)),
          "rope_cache");
  });
  m.def("kv_write", [](uptr k, uptr v, long stride, uptr slots, int T, int Hkv, int D, uptr kc,
                       uptr vc, int BS, uptr stream) {
    check(lmx::kv_write(P<void>(k), P<void>(v), stride, P<int>(slots), T, Hkv, D, P<void>(kc),
                        P<void>(vc), BS, S(stream)),
          "kv_write");
  });
  m.def("paged_decode", [](uptr q, long q_stride, uptr kc, uptr vc, uptr bt, int bt_stride,
                           uptr ctx, uptr order, uptr out, long out_stride, uptr part_o,
                           uptr part_ml, int B, int Hq, int Hkv, int D, int BS, float scale,
                           int part_tokens, int max_parts, uptr positions, uptr cos_sin,
                           uptr slots, uptr gate, long gate_stride, int split_p, int window,
                           float cap, uptr stream) {
    check(lmx::paged_decode(P<void>(q), q_stride, P<void>(kc), P<void>(vc), P<int>(bt), bt_stride,
                            P<int>(ctx), P<int>(order), P<void>(out), out_stride, P<float>(part_o),
                            P<float>(part_ml), B, Hq, Hkv, D, BS, scale, part_tokens, max_parts,
                            P<int>(positions), P<float>(cos_sin), P<int>(slots), P<void>(gate),
                            gate_stride, split_p, window, cap, S(stream)),
          "paged_decode");
  });
  m.def("set_slab_norm_threads", [](int t) { lmx::set_slab_norm_threads(t); },
        "probe knob: workgroup size cap of the slab RMSNorm (default 512)");
  m.def("set_decode_mode", [](int mode) { lmx::set_decode_mode(mode); },
        "paged decode loop: 0 one page at a time, 1 next page prefetched, 2 loads only (probe)");
  m.def("set_prefill_rescale_thr", [](float thr) { lmx::set_prefill_rescale_thr(thr); },
        "prefill softmax: raise the running max only past this many log2 units (0: always)");
  m.def("set_prefill_stages", [](int n) { lmx::set_prefill_stages(n); },
        "prefill attention LDS ring slots: 0 default per head dim, 2 or 3");
  m.def("set_prefill_xcd", [](int on) { lmx::set_prefill_xcd(on); },
        "prefill attention workgroup order: 2 XCD-aware, tile list reversed (default), 1 XCD-aware, 0 hardware order");
  m.def("paged_prefill", [](uptr q, long q_stride, uptr kc, uptr vc, uptr bt, int bt_stride,
                            uptr cu_q, uptr ctx, uptr tiles, int num_tiles, uptr out,
                            long out_stride, int Hq, int Hkv, int D, int BS, float scale,
                            int causal, int q_per_tile, uptr rope_pos, uptr rope_cs, uptr gate,
                            long gate_stride, int split_p, int window, float cap,
                            uptr stream) {
    check(lmx::paged_prefill(P<void>(q), q_stride, P<void>(kc), P<void>(vc), P<int>(bt),
                             bt_stride, P<int>(cu_q), P<int>(ctx), P<int>(tiles), num_tiles,
                             P<void>(out), out_stride, Hq, Hkv, D, BS, scale, causal, q_per_tile,
                             P<int>(rope_pos), P<float>(rope_cs), P<void>(gate), gate_stride,
                             split_p, window, cap, S(stream)),
          "paged_prefill");
  });
  m.def("attention_any", [](uptr q, long q_stride, uptr kc, uptr vc, uptr bt, int bt_stride,
                            uptr cu_q, int nseq, uptr positions, int rows, uptr out,
                            long out_stride, uptr gate, long gate_stride, int Hq, int Hkv, int D,
                            int BS, float scale, int window, float cap, int is_bf16,
                            uptr stream) {
    check(lmx::attention_any(P<void>(q), q_stride, P<void>(kc), P<void>(vc), P<int>(bt), bt_stride,
                             P<int>(cu_q), nseq, P<int>(positions), rows, P<void>(out), out_stride,
                             P<void>(gate), gate_stride, Hq, Hkv, D, BS, scale, window, cap,
                             is_bf16, S(stream)),
          "attention_any");
  });
  // ---- sandwich / gated norms (norm.hip) ----
  m.def("sandwich_norm", [](uptr out, uptr residual, uptr y, long y_ld, int slabs,
                            long slab_stride, uptr mix_pos, uptr mix_w, int mix_n, uptr own,
                            uptr bias, uptr ids, uptr table, float scale, uptr w_post, uptr w_pre, uptr rows_idx, int rows, int cols, float eps, int is_bf16,
                            uptr stream) {
    check(lmx::sandwich_norm(P<void>(out), P<float>(residual), P<void>(y), y_ld, slabs,
                             slab_stride, P<int>(mix_pos), P<float>(mix_w), mix_n, P<float>(own),
                             P<float>(bias), P<int>(ids), P<void>(table), scale, P<float>(w_post), P<float>(w_pre), P<long>(rows_idx), rows, cols, eps, is_bf16,
                             S(stream)),
          "sandwich_norm");
  });
  m.def("sum_norm", [](uptr out, uptr residual, uptr ya, long a_ld, int a_slabs, long a_stride,
                       uptr mix_pos, uptr mix_w, int mix_n, uptr yb, long b_ld, int b_slabs,
                       long b_stride, uptr wa, uptr wb, float alpha, uptr scale, uptr w_post,
                       uptr w_pre, uptr rows_idx, int rows, int cols, float eps, int is_bf16,
                       uptr stream) {
    check(lmx::sum_norm(P<void>(out), P<float>(residual), P<void>(ya), a_ld, a_slabs, a_stride,
                        P<int>(mix_pos), P<float>(mix_w), mix_n, P<void>(yb), b_ld, b_slabs,
                        b_stride, P<float>(wa), P<float>(wb), alpha, P<float>(scale),
                        P<float>(w_post), P<float>(w_pre), P<long>(rows_idx), rows, cols, eps,
                        is_bf16, S(stream)),
          "sum_norm");
  });
  m.def("soft_cap", [](uptr x, long n, float scale, float cap, int is_bf16, uptr stream) {
    check(lmx::soft_cap(P<void>(x), n, scale, cap, is_bf16, S(stream)), "soft_cap");
  });
  m.def("rotate_rows", [](uptr q, long q_ld, uptr k, long k_ld, uptr ang, int n, int r0, int r1,
                          int groups, int N, float k_scale, uptr stream) {
    check(lmx::rotate_rows(P<void>(q), q_ld, P<void>(k), k_ld, P<float>(ang), n, r0, r1, groups, N,
                           k_scale, S(stream)),
          "rotate_rows");
  });
  m.def("norm_rope_cache", [](uptr p, long p_ld, uptr q_norm, uptr k_norm, uptr ang, int n,
                              uptr slots, uptr quads, int groups, uptr q, uptr kc, uptr vc, int Hq,
                              int Hkv, int D, int dk, int BS, float eps, int is_bf16, uptr stream) {
    check(lmx::norm_rope_cache(P<void>(p), p_ld, P<float>(q_norm), P<float>(k_norm), P<float>(ang),
                               n, P<int>(slots), P<int>(quads), groups, P<void>(q), P<void>(kc),
                               P<void>(vc), Hq, Hkv, D, dk, BS, eps, is_bf16, S(stream)),
          "norm_rope_cache");
  });
  // ---- K21 gated delta rule (delta.hip) ----
  m.def("delta_recurrent", [](uptr q, long q_ld, uptr k, long k_ld, uptr v, long v_ld, uptr b,
                              long b_ld, uptr a, long a_ld, uptr dt_bias, uptr neg_a, uptr out,
                              long out_ld, uptr state, uptr cu_q, uptr ctx, uptr slots, int H,
                              int G, int N, int Pd, int nseq, int is_bf16, uptr stream) {
    const lmx::DeltaArgs d{P<void>(q), P<void>(k), P<void>(v), P<void>(b), P<void>(a), q_ld, k_ld,
                           v_ld, b_ld, a_ld, P<float>(dt_bias), P<float>(neg_a), P<void>(out),
                           out_ld, P<float>(state), P<int>(cu_q), P<int>(ctx), P<int>(slots), H, G,
                           N, Pd};
    check(lmx::delta_recurrent(d, nseq, is_bf16, S(stream)), "delta_recurrent");
  });
  m.def("delta_chunks", [](uptr q, long q_ld, uptr k, long k_ld, uptr v, long v_ld, uptr b,
                           long b_ld, uptr a, long a_ld, uptr dt_bias, uptr neg_a, uptr out,
                           long out_ld, uptr state, uptr cu_q, uptr ctx, uptr slots, int H, int G,
                           int N, int Pd, int seq0, int nseq, uptr chunks, int nchunks, uptr first,
                           uptr mats, uptr vecs, uptr stream) {
    const lmx::DeltaArgs d{P<void>(q), P<void>(k), P<void>(v), P<void>(b), P<void>(a), q_ld, k_ld,
                           v_ld, b_ld, a_ld, P<float>(dt_bias), P<float>(neg_a), P<void>(out),
                           out_ld, P<float>(state), P<int>(cu_q), P<int>(ctx), P<int>(slots), H, G,
                           N, Pd};
    check(lmx::delta_chunks(d, seq0, nseq, P<int>(chunks), nchunks, P<int>(first), P<void>(mats),
                            P<float>(vecs), S(stream)),
          "delta_chunks");
  });
  m.def("gelu", [](uptr x, long n, int is_bf16, uptr stream) {
    check(lmx::gelu(P<void>(x), n, is_bf16, S(stream)), "gelu");
  });
  m.def("grouped", [](uptr a, long lda, long a_gs, uptr w, uptr c, long ldc, long c_gs, int groups,
                      int N, int K, int M, uptr tiles, int mtiles, uptr off, uptr src, uptr limit,
                      float slope, float shift, uptr gate, long gate_ld, int bm, int is_bf16,
                      uptr stream) {
    check(lmx::grouped(P<void>(a), lda, a_gs, P<void>(w), P<void>(c), ldc, c_gs, groups, N, K, M,
                       P<int>(tiles), mtiles, P<int>(off), P<int>(src), P<float>(limit), slope,
                       shift, P<void>(gate), gate_ld, bm, is_bf16, S(stream)),
          "grouped");
  });
  m.def("pgemm_grouped", [](uptr c, uptr a, uptr w, int M, int N, int K, long lda, long ldc,
                            int a_rows, uptr tiles, int mtiles, uptr off, uptr src, uptr limit,
                            float slope, float shift, uptr stream) {
    check(lmx::pgemm_grouped(P<void>(c), P<void>(a), P<void>(w), M, N, K, lda, ldc, a_rows,
                             P<int>(tiles), mtiles, P<int>(off), P<int>(src), P<float>(limit),
                             slope, shift, S(stream)),
          "pgemm_grouped");
  });
  m.def("moe_route", [](uptr h, long h_ld, uptr w, int T, int d, int E, int rows, int top,
                        int extra, uptr correction, int groups, int keep, int softmax, int identity,
                        uptr ids, uptr wts, uptr own, int is_bf16, uptr stream) {
    check(lmx::moe_route(P<void>(h), h_ld, P<void>(w), T, d, E, rows, top, extra,
                         P<float>(correction), groups, keep, softmax, identity, P<int>(ids),
                         P<float>(wts), P<float>(own), is_bf16, S(stream)),
          "moe_route");
  });
  m.def("bias_relu2", [](uptr x, uptr bias, long rows, int cols, int is_bf16, uptr stream) {
    check(lmx::bias_relu2(P<void>(x), P<float>(bias), rows, cols, is_bf16, S(stream)), "bias_relu2");
  });
  // ---- K22 talking heads (talk.hip) ----
  m.def("qkv_norm_rope_cache", [](uptr p, long p_ld, uptr bias, uptr q_norm, uptr k_norm, uptr ang,
                                  int n, uptr slots, uptr quads, int groups, uptr q, uptr kc, uptr vc,
                                  int Hq, int Hkv, int D, int dk, int dv, int BS, float eps,
                                  int is_bf16, uptr stream) {
    check(lmx::qkv_norm_rope_cache(P<void>(p), p_ld, P<float>(bias), P<float>(q_norm),
                                   P<float>(k_norm), P<float>(ang), n, P<int>(slots), P<int>(quads),
                                   groups, P<void>(q), P<void>(kc), P<void>(vc), Hq, Hkv, D, dk, dv,
                                   BS, eps, is_bf16, S(stream)),
          "qkv_norm_rope_cache");
  });
  m.def("talk_prefill", [](uptr q, uptr kc, uptr vc, uptr mix, uptr sink, float out_scale, int Hq,
                           int Hkv, int D, int chunk, uptr bt, int bt_stride, uptr cu_q, uptr ctx,
                           uptr tiles, int n, uptr gate, long gate_ld, uptr out, long out_ld,
                           uptr stream) {
    check(lmx::talk_prefill(P<void>(q), P<void>(kc), P<void>(vc), P<void>(mix), P<float>(sink),
                            out_scale, Hq, Hkv, D, chunk, P<int>(bt), bt_stride, P<int>(cu_q),
                            P<int>(ctx), P<int>(tiles), n, P<void>(gate), gate_ld, P<void>(out),
                            out_ld, S(stream)),
          "talk_prefill");
  });
  m.def("talk_decode", [](uptr q, uptr kc, uptr vc, uptr mix, uptr sink, float out_scale, int Hq,
                          int Hkv, int D, int chunk, uptr bt, int bt_stride, uptr ctx, int rows,
                          uptr gate, long gate_ld, uptr out, long out_ld, uptr part_o, uptr part_ml,
                          int part_tokens, int max_parts, uptr stream) {
    check(lmx::talk_decode(P<void>(q), P<void>(kc), P<void>(vc), P<void>(mix), P<float>(sink),
                           out_scale, Hq, Hkv, D, chunk, P<int>(bt), bt_stride, P<int>(ctx), rows,
                           P<void>(gate), gate_ld, P<void>(out), out_ld, P<float>(part_o),
                           P<float>(part_ml), part_tokens, max_parts, S(stream)),
          "talk_decode");
  });
  m.def("talk_any", [](uptr q, uptr kc, uptr vc, uptr bt, int bt_stride, uptr cu_q, int nseq,
                       uptr positions, int rows, uptr mix, uptr sink, uptr out, long out_ld, uptr gate,
                       long gate_ld, float out_scale, int Hq, int Hkv, int D, int chunk, int is_bf16,
                       uptr stream) {
    check(lmx::talk_any(P<void>(q), P<void>(kc), P<void>(vc), P<int>(bt), bt_stride, P<int>(cu_q),
                        nseq, P<int>(positions), rows, P<void>(mix), P<float>(sink), P<void>(out),
                        out_ld, P<void>(gate), gate_ld, out_scale, Hq, Hkv, D, chunk, is_bf16,
                        S(stream)),
          "talk_any");
  });
  // ---- K15 matrix memory (linscan.hip) ----
  m.def("memory_scan", [](uptr q, long q_ld, uptr k, long k_ld, uptr v, long v_ld, uptr ig, uptr fg,
                          long gate_ld, uptr gate_bias, float cap, uptr out, long out_ld, uptr state,
                          uptr sn, uptr sm, uptr cu_q, uptr ctx, uptr slots, int H, int N, int Pd,
                          int is_bf16, int seq0, int nseq, uptr segs, int nseg, uptr first,
                          int one_pass, uptr ws, uptr ws_n, uptr stream) {
    check(lmx::memory_scan(P<void>(q), q_ld, P<void>(k), k_ld, P<void>(v), v_ld, P<void>(ig),
                           P<void>(fg), gate_ld, P<float>(gate_bias), cap, P<void>(out), out_ld,
                           P<float>(state), P<float>(sn), P<float>(sm), P<int>(cu_q), P<int>(ctx),
                           P<int>(slots), H, N, Pd, is_bf16, seq0, nseq, P<int>(segs), nseg,
                           P<int>(first), one_pass, P<float>(ws), P<float>(ws_n), S(stream)),
          "memory_scan");
  });
  m.def("moe_plan", [](uptr ids, int n, int J, int groups, int bm, int mtiles, uptr hist, uptr off,
                       uptr src, uptr pos, uptr tiles, uptr stream) {
    check(lmx::moe_plan(P<int>(ids), n, J, groups, bm, mtiles, P<int>(hist), P<int>(off),
                        P<int>(src), P<int>(pos), P<int>(tiles), S(stream)),
          "moe_plan");
  });
  m.def("rglru_chunks", [](uptr u, uptr y, long y_ld, uptr y_b, uptr g_b, uptr log_a, uptr out,
                           uptr state, uptr cu_q, uptr ctx, uptr slots, int C, int bp, uptr w,
                           int seq0, uptr segs, int nsegs, uptr first, uptr ws, uptr stream) {
    check(lmx::rglru_chunks(P<void>(u), P<void>(y), y_ld, P<float>(y_b), P<float>(g_b),
                            P<float>(log_a), P<void>(out), P<float>(state), P<int>(cu_q),
                            P<int>(ctx), P<int>(slots), C, bp, P<void>(w), seq0, P<int>(segs), nsegs,
                            P<int>(first), P<float>(ws), S(stream)),
          "rglru_chunks");
  });
  m.def("rglru_rows", [](uptr u, uptr y, long y_ld, uptr y_b, uptr g_b, uptr log_a, uptr out,
                         uptr state, uptr cu_q, uptr ctx, uptr slots, int C, int bp, uptr w,
                         int rows, uptr stream) {
    check(lmx::rglru_rows(P<void>(u), P<void>(y), y_ld, P<float>(y_b), P<float>(g_b),
                          P<float>(log_a), P<void>(out), P<float>(state), P<int>(cu_q), P<int>(ctx),
                          P<int>(slots), C, bp, P<void>(w), rows, S(stream)),
          "rglru_rows");
  });
  m.def("rglru_scan", [](uptr u, uptr y, long y_ld, uptr y_b, uptr g_b, uptr log_a, uptr out,
                         uptr state, uptr cu_q, uptr ctx, uptr slots, int C, int bp, uptr z, int nseq,
                         int is_bf16, uptr stream) {
    check(lmx::rglru_scan(P<void>(u), P<void>(y), y_ld, P<float>(y_b), P<float>(g_b),
                          P<float>(log_a), P<void>(out), P<float>(state), P<int>(cu_q), P<int>(ctx),
                          P<int>(slots), C, bp, P<float>(z), nseq, is_bf16, S(stream)),
          "rglru_scan");
  });
  m.def("rope_angles", [](uptr positions, uptr freqs, int T, int n, float scale, uptr out,
                          uptr stream) {
    check(lmx::rope_angles(P<int>(positions), P<double>(freqs), T, n, scale, P<float>(out),
                           S(stream)),
          "rope_angles");
  });
  m.def("latent_prep", [](uptr p, long p_ld, int T, int qr, int qp, uptr q_norm, int R, int Rp,
                          uptr c_norm, uptr ang, int d, uptr slots, uptr pages, int BS, int D,
                          uptr cq, float eps, int is_bf16, uptr stream) {
    check(lmx::latent_prep(P<void>(p), p_ld, T, qr, qp, P<float>(q_norm), R, Rp, P<float>(c_norm),
                           P<float>(ang), d, P<int>(slots), P<void>(pages), BS, D, P<void>(cq), eps,
                           is_bf16, S(stream)),
          "latent_prep");
  });
  m.def("latent_rotate", [](uptr q, long q_ld, int np, uptr ang, int d, int T, int H, int xp,
                            uptr out, long o_ld, int Rp, int is_bf16, uptr stream) {
    check(lmx::latent_rotate(P<void>(q), q_ld, np, P<float>(ang), d, T, H, xp, P<void>(out), o_ld,
                             Rp, is_bf16, S(stream)),
          "latent_rotate");
  });
  m.def("latent_any", [](uptr q, uptr pages, uptr bt, int bt_stride, uptr cu_q, int nseq,
                         uptr positions, int rows, uptr out, int H, int Rp, int D, float scale,
                         int window, int is_bf16, uptr stream) {
    check(lmx::latent_any(P<void>(q), P<void>(pages), P<int>(bt), bt_stride, P<int>(cu_q), nseq,
                          P<int>(positions), rows, P<void>(out), H, Rp, D, scale, window, is_bf16,
                          S(stream)),
          "latent_any");
  });
  m.def("latent_gather", [](uptr pages, uptr bt, int bt_stride, uptr seqs, int nseq, int n, int D,
                            uptr out, uptr stream) {
    check(lmx::latent_gather(P<void>(pages), P<int>(bt), bt_stride, P<int>(seqs), nseq, n, D,
                             P<void>(out), S(stream)),
          "latent_gather");
  });
  m.def("latent_prefill", [](uptr q, long q_ld, uptr kv, uptr lat, uptr ang, uptr seqs, uptr tiles,
                             int ntiles, uptr cu_q, uptr ctx, uptr gate, long gate_ld, uptr out,
                             long out_ld, int H, int NP, int VP, int D, int Rp, int d, float scale,
                             int window, uptr stream) {
    check(lmx::latent_prefill(P<void>(q), q_ld, P<void>(kv), P<void>(lat), P<float>(ang),
                              P<int>(seqs), P<int>(tiles), ntiles, P<int>(cu_q), P<int>(ctx),
                              P<void>(gate), gate_ld, P<void>(out), out_ld, H, NP, VP, D, Rp, d,
                              scale, window, S(stream)),
          "latent_prefill");
  });
  m.def("latent_rows", [](uptr q, uptr pages, uptr bt, int bt_stride, uptr cu_q, int nseq,
                          uptr positions, int rows, int num_decode, uptr out, uptr part_o,
                          uptr part_ml, int H, int Rp, int D, float scale, int window,
                          int part_keys, int max_parts, uptr stream) {
    check(lmx::latent_rows(P<void>(q), P<void>(pages), P<int>(bt), bt_stride, P<int>(cu_q), nseq,
                           P<int>(positions), rows, num_decode, P<void>(out), P<float>(part_o),
                           P<float>(part_ml), H, Rp, D, scale, window, part_keys, max_parts,
                           S(stream)),
          "latent_rows");
  });
  m.def("gated_norm", [](uptr out, long out_ld, uptr x, long x_ld, uptr g, long g_ld, uptr w,
                         int rows, int cols, int groups, int gate_first, float eps, int is_bf16,
                         uptr stream) {
    check(lmx::gated_norm(P<void>(out), out_ld, P<void>(x), x_ld, P<void>(g), g_ld, P<float>(w),
                          rows, cols, groups, gate_first, eps, is_bf16, S(stream)),
          "gated_norm");
  });
  // ---- K16 short causal convolution (conv.hip) ----
  m.def("short_conv", [](uptr u, long u_ld, uptr w, uptr in_bias, uptr bias, uptr state, uptr tiles,
                         int ntiles, int tile, uptr cu_q, uptr ctx, uptr slots, int C, int taps, uptr out,
                         long out_ld, int act, int is_bf16, uptr stream) {
    check(lmx::short_conv(P<void>(u), u_ld, P<float>(w), P<float>(in_bias), P<float>(bias), P<void>(state),
                          P<int>(tiles), ntiles, tile, P<int>(cu_q), P<int>(ctx), P<int>(slots), C,
                          taps, P<void>(out), out_ld, act, is_bf16, S(stream)),
          "short_conv");
  });
  m.def("conv_qkv_cache", [](uptr u, long u_ld, uptr w, uptr in_bias, uptr state, uptr tiles,
                             int ntiles, int tile, uptr cu_q, uptr ctx, uptr state_slots, int taps, uptr q,
                             long q_ld, uptr kc, uptr vc, uptr positions, uptr slots, int Hq,
                             int Hkv, int D, int dk, int BS, float eps, float coef, float every,
                             int is_bf16, uptr stream) {
    check(lmx::conv_qkv_cache(P<void>(u), u_ld, P<float>(w), P<float>(in_bias), P<void>(state),
                              P<int>(tiles), ntiles, tile, P<int>(cu_q), P<int>(ctx), P<int>(state_slots), taps,
                              P<void>(q), q_ld, P<void>(kc), P<void>(vc), P<int>(positions),
                              P<int>(slots), Hq, Hkv, D, dk, BS, eps, coef, every, is_bf16,
                              S(stream)),
          "conv_qkv_cache");
  });
  // ---- K15 linear-attention / state-space scan (linscan.hip) ----
  m.def("linear_scan", [](uptr q, long q_ld, uptr k, long k_ld, uptr v, long v_ld, uptr dt,
                          long dt_ld, uptr dt_bias, uptr neg_a, uptr decay, uptr log_decay,
                          uptr skip, uptr out, long out_ld, uptr state, uptr cu_q, uptr ctx,
                          uptr slots, int H, int N, int Pd, int hpg, int act, int is_bf16,
                          uptr ang, int nrot, float k_scale, int seq0,
                          int nseq, uptr segs, int nseg, uptr first, int one_pass, uptr ws,
                          uptr ws_log, uptr stream) {
    check(lmx::linear_scan(P<void>(q), q_ld, P<void>(k), k_ld, P<void>(v), v_ld, P<void>(dt),
                           dt_ld, P<float>(dt_bias), P<float>(neg_a), P<float>(decay),
                           P<float>(log_decay), P<float>(skip), P<void>(out), out_ld,
                           P<float>(state), P<int>(cu_q), P<int>(ctx), P<int>(slots), H, N, Pd, hpg,
                           act, is_bf16, P<float>(ang), nrot, k_scale, seq0, nseq, P<int>(segs), nseg, P<int>(first), one_pass,
                           P<float>(ws), P<float>(ws_log), S(stream)),
          "linear_scan");
  });
  m.def("sample", [](uptr logits, int is_bf16, long stride, int B, int V, uptr temp, uptr topk,
                     uptr topp, uptr seeds, uptr offsets, uptr out_tok, uptr out_lp,
                     int max_rounds, uptr stream) {
    check(lmx::sample(P<void>(logits), is_bf16, stride, B, V, P<float>(temp), P<int>(topk),
                      P<float>(topp), P<uint64_t>(seeds), P<int>(offsets), P<int>(out_tok),
                      P<float>(out_lp), max_rounds, S(stream)),
          "sample");
  });
  m.def("glu", [](uptr out, uptr x, long rows, int I, int act, int block, int is_bf16,
                  uptr stream) {
    check(lmx::glu(P<void>(out), P<void>(x), rows, I, act, block, is_bf16, S(stream)), "glu");
  });
  m.def("ids_from_prev", [](uptr ids, uptr src, uptr prev, int n, uptr stream) {
    check(lmx::ids_from_prev(P<int>(ids), P<int>(src), P<int>(prev), n, S(stream)),
          "ids_from_prev");
  });
  m.def("embed_gather", [](uptr out, uptr table, uptr ids, int T, int d, int vs, int vr,
                           uptr stream) {
    check(lmx::embed_gather(P<void>(out), P<void>(table), P<int>(ids), T, d, vs, vr, S(stream)),
          "embed_gather");
  });
  m.def("mean_pool_l2", [](uptr out, uptr acc, uptr h, uptr cu, int nseq, int T, int d, int dims,
                           int norm, uptr stream) {
    check(lmx::mean_pool_l2(P<float>(out), P<float>(acc), P<void>(h), P<int>(cu), nseq, T, d, dims,
                            norm, S(stream)),
          "mean_pool_l2");
  });
  m.def("bias_act", [](uptr x, uptr bias, long rows, int n, int act, uptr stream) {
    check(lmx::bias_act(P<void>(x), P<void>(bias), rows, n, act, S(stream)), "bias_act");
  });
  m.def("gemm_splitk", [](uptr C, uptr A, uptr W, uptr slabs, uptr tickets, int M, int N, int K,
                          long lda, long ldw, long ldc, int splits, uptr stream) {
    check(lmx::gemm_splitk(P<void>(C), P<void>(A), P<void>(W), P<float>(slabs), P<int>(tickets), M,
                           N, K, lda, ldw, ldc, splits, S(stream)),
          "gemm_splitk");
  });
  m.def("dgemm", [](uptr C, uptr A, uptr W, uptr slabs, uptr tickets, int n_tickets, int M, int N,
                    int K, long lda, long ldw, long ldc, int cfg, int splits, int epi,
                    uptr stream) {
    check(lmx::dgemm(P<void>(C), P<void>(A), P<void>(W), P<float>(slabs), P<unsigned>(tickets),
                     n_tickets, M, N, K, lda, ldw, ldc, cfg, splits, epi, S(stream)),
          "dgemm");
  });
  m.def("rmsnorm_slabs", [](uptr out, uptr residual, uptr slabs, int nsl, long slab_stride,
                            uptr w, int rows, int cols, long out_stride, float eps, uptr stream) {
    check(lmx::rmsnorm_slabs(P<void>(out), P<void>(residual), P<float>(slabs), nsl, slab_stride,
                             P<void>(w), rows, cols, out_stride, eps, S(stream)),
          "rmsnorm_slabs");
  });
  m.def("dgemm_sk_pieces", [](int M, int N, int K, int cfg, int groups) {
    return lmx::dgemm_sk_pieces(M, N, K, cfg, groups);
  });
  m.def("dgemm_configs", []() {
    std::vector<std::pair<int, int>> out;
    for (int i = 0; i < lmx::dgemm_num_configs(); ++i) {
      int bm = 0, bn = 0;
      lmx::dgemm_config(i, &bm, &bn);
      out.emplace_back(bm, bn);
    }
    return out;
  });
  // ---- K14 register-streamed decode GEMM (rsgemm.hip) ----
  m.def("rsgemm", [](uptr C, uptr A, uptr Wp, uptr slabs, uptr tickets, int n_tickets, int M, int N,
                     int K, long lda, long ldw, long ldc, int cfg, int splits, int epi,
                     uptr stream) {
    check(lmx::rsgemm(P<void>(C), P<void>(A), P<void>(Wp), P<float>(slabs), P<unsigned>(tickets),
                      n_tickets, M, N, K, lda, ldw, ldc, cfg, splits, epi, S(stream)),
          "rsgemm");
  });
  m.def("rsgemm_pack", [](uptr out, uptr W, int N, int K, long ldw, uptr stream) {
    check(lmx::rsgemm_pack(P<void>(out), P<void>(W), N, K, ldw, S(stream)), "rsgemm_pack");
  });
  // ---- K13 large-M GEMM (pgemm.hip) ----
  m.def("pgemm", [](uptr C, uptr A, uptr W, uptr bias, int M, int N, int K, long lda, long ldw,
                    long ldc, int act, int grid, int res, int wpacked, uptr nrm, uptr stream) {
    check(lmx::pgemm(P<void>(C), P<void>(A), P<void>(W), P<void>(bias), M, N, K, lda, ldw, ldc,
                     act, grid, res, wpacked, P<float>(nrm), S(stream)),
          "pgemm");
  });
  m.def("row_scale", [](uptr s, uptr part, int np, uptr x, long x_stride, int M, int cols,
                        float eps, uptr stream) {
    check(lmx::row_scale(P<float>(s), P<float>(part), np, P<void>(x), x_stride, M, cols, eps,
                         S(stream)),
          "row_scale");
  }, "RMSNorm row scales rsqrt(mean(x^2) + eps): from fp32 partials [M][P] or bf16 rows x");
  m.def("pgemm_sk", [](uptr C, uptr A, uptr W, uptr slabs, uptr cnt, int n_cnt, int M, int N,
                       int K, long lda, long ldw, long ldc, int act, int splits, int epi,
                       uptr stream) {
    check(lmx::pgemm_sk(P<void>(C), P<void>(A), P<void>(W), P<void>(slabs), P<void>(cnt), n_cnt,
                        M, N, K, lda, ldw, ldc, act, splits, epi, S(stream)),
          "pgemm_sk");
  });
  // ---- peer-memory all-reduce (allreduce.hip) ----
  m.def("ar_region_bytes", [](long slot) { return lmx::ar_region_bytes(slot); });
  m.def("ar_alloc", [](long slot) {
    void* p = nullptr;
    check(lmx::ar_alloc(&p, slot), "ar_alloc");
    return (uptr)p;
  });
  m.def("ar_free", [](uptr p) { check(lmx::ar_free(P<void>(p)), "ar_free"); });
  m.def("ar_ipc_handle", [](uptr p) {
    std::string h((size_t)lmx::ar_ipc_handle_size(), '\0');
    check(lmx::ar_ipc_handle(P<void>(p), h.data()), "ar_ipc_handle");
    return py::bytes(h);
  });
  m.def("ar_ipc_open", [](py::bytes handle) {
    std::string h = handle;
    if ((int)h.size() != lmx::ar_ipc_handle_size())
      throw std::runtime_error("ar_ipc_open: bad handle size");
    void* p = nullptr;
    check(lmx::ar_ipc_open(&p, h.data()), "ar_ipc_open");
    return (uptr)p;
  });
  m.def("ar_ipc_close", [](uptr p) { check(lmx::ar_ipc_close(P<void>(p)), "ar_ipc_close"); });
  m.def("ar_error", [](uptr own, int clear) {
    const int v = lmx::ar_error(P<void>(own), clear);
    if (v < 0) check(-v, "ar_error");
    return v;
  });
  m.def("allreduce_norm", [](uptr h_out, uptr residual, uptr inp, uptr w, int T, int cols,
                             float eps, int rank, int world, std::vector<unsigned long long> peers,
                             long slot_bytes, int two_shot, int groups, int cs, int spin_max,
                             uptr stream) {
    if ((int)peers.size() < world) throw std::runtime_error("allreduce_norm: peers < world");
    check(lmx::allreduce_norm(P<void>(h_out), P<void>(residual), P<void>(inp), P<void>(w), T,
                              cols, eps, rank, world, peers.data(), slot_bytes, two_shot, groups,
                              cs, spin_max, S(stream)),
          "allreduce_norm");
  });
  m.def("ar_error_async", [](uptr own, uptr host, uptr stream) {
    check(lmx::ar_error_async(P<void>(own), P<void>(host), S(stream)), "ar_error_async");
  });
  m.def("allreduce", [](uptr out, uptr inp, long nbytes, int rank, int world,
                        std::vector<unsigned long long> peers, long slot_bytes, int two_shot,
                        int blocks, int spin_max, uptr stream) {
    if ((int)peers.size() < world) throw std::runtime_error("allreduce: peers < world");
    check(lmx::allreduce(P<void>(out), P<void>(inp), nbytes, rank, world, peers.data(), slot_bytes,
                         two_shot, blocks, spin_max, S(stream)),
          "allreduce");
  });
  m.def("apply_penalties", [](uptr logits, int is_bf16, long ld, int B, int V, uptr win, uptr ngen, uptr pen,
                              uptr on, int W, int v0, uptr stream) {
    check(lmx::apply_penalties(P<void>(logits), is_bf16, ld, B, V, P<const int>(win), P<const int>(ngen),
                               P<const float>(pen), P<const int>(on), W, v0, S(stream)),
          "apply_penalties");
  });
  m.def("race_sample_phase", [](int phase, int round, int max_rounds, uptr logits, int is_bf16,
                                long stride, int B, int Vs, int v0, int V, uptr temp, uptr topk,
                                uptr topp, uptr seeds, uptr offsets, uptr gath, int W, uptr rec,
                                uptr st, uptr out_tok, uptr out_lp, uptr stream) {
    check(lmx::race_sample_phase(phase, round, max_rounds, P<void>(logits), is_bf16, stride, B, Vs,
                                 v0, V, P<float>(temp), P<int>(topk), P<float>(topp),
                                 P<uint64_t>(seeds), P<int>(offsets), P<float>(gath), W,
                                 P<float>(rec), P<float>(st), P<int>(out_tok), P<float>(out_lp),
                                 S(stream)),
          "race_sample_phase");
  });
  m.def("gemm_nt", [](uptr C, uptr A, uptr W, uptr bias, uptr residual, int M, int N, int K,
                      long lda, long ldw, long ldc, int act, uptr stream) {
    check(lmx::gemm_nt(P<void>(C), P<void>(A), P<void>(W), P<void>(bias), P<void>(residual), M, N,
                       K, lda, ldw, ldc, act, S(stream)),
          "gemm_nt");
  });
}
