// Parameters of the generalised delta rule's kernels (csrc/hybrid/channel_delta*.hip).
#pragma once
#include "hybrid.h"

namespace nxd {

struct ChannelDeltaParams {
  int B, T;                  // sequences, new tokens per sequence (row b * T + t)
  int H, D, DP, N;           // heads, head size, D rounded up to 32, rank of the decay's projection
  const void* proj;          // [B T, ldp] r | k | v | gate | removal (H D each) | low (N)
  int64_t ldp;
  const void* w2;            // [H D, N] (activation type)
  const float *w0, *a_bias, *norm_w;   // [H D]
  float eps, out_scale;
  const int64_t* pos;        // position of each sequence's first new token: pos[b * pos_stride]
  int64_t pos_stride;
  const int* lens;           // [B] valid new tokens (nullable: T)
  const int* slots;          // [B] cache slots (nullable: identity)
  int nslots;
  float* state;              // [slots, H, D (value), DP (key)]
  void* y;                   // [B T, ldy] output before the projection (activation type)
  int64_t ldy;
  // chunks (channel_delta_chunk.hip), a cell = (sequence, chunk, head)
  int nch;
  float *cq, *co, *cw, *cy, *cb, *ck, *cv;   // Q, O', W, Y, E B^T, E K^T, V [cells, C DP]
  float *cs, *ce;            // S_0 [cells, DP DP], E [cells, DP]
};

namespace hybrid {

// log2 of the decay from the projection's output x: -e^(-1/2) sigmoid(x) / ln 2
__device__ __forceinline__ float decay_log2(float x) { return -0.8750387749145276f / (1.f + expf(-x)); }

__device__ __forceinline__ float tanhf_(float x) {   // 1 - 2 / (1 + e^(2 x)); small x by its series
  const float a = fabsf(x);
  if (a < 0.05f) return x * (1.f - x * x * (1.f / 3.f - x * x * (2.f / 15.f)));
  const float t = 1.f - 2.f / (1.f + expf(2.f * a));
  return x < 0.f ? -t : t;
}

}  // namespace hybrid
}  // namespace nxd
