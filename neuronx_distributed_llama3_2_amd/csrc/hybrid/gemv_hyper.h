// Parameters of the fused decode projections (csrc/hybrid/gemv_hyper.hip).
#pragma once
#include "hybrid.h"

namespace nxd {

struct GemvHyperParams {
  const uint16_t* x;      // [M, K] bf16 (no norm)
  int64_t ldx;
  const float* u;         // [M, K] fp32 (norm)
  const float* norm_w;    // [K]
  float eps;
  const uint16_t* w;      // [N, K]
  int64_t ldw;
  int M, N, K;
  void* y;                // [M, N]
  int64_t ldy;
  float alpha, cap;       // fp32 outputs: cap tanh(alpha y / cap), or alpha y
  // HYPER
  float* streams;         // [M, S, N]
  int S;
  const float *bias, *mix, *write, *read;
  float* un;              // [M, N]
};

}  // namespace nxd
