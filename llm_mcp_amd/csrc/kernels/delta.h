// Operands of the gated delta rule (delta.hip).
#pragma once

namespace lmx {

struct DeltaArgs {
  const void *q, *k, *v, *b, *a;   // rows: G x N, G x N, H x P channels, H, H values
  long q_ld, k_ld, v_ld, b_ld, a_ld;
  const float *dt_bias, *neg_a;    // [H]
  void* out;                       // rows of H x P
  long out_ld;
  float* state;                    // [slots][H][N][P]
  const int *cu_q, *ctx, *slots;
  int H, G, N, P;
};

}  // namespace lmx
