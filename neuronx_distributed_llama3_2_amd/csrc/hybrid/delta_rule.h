// Parameters of the gated-delta-rule kernels (csrc/hybrid/delta_rule.hip) and of their launchers.
#pragma once
#include "hybrid.h"

namespace nxd {

struct DeltaParams {
  int B, T;                  // sequences, new tokens per sequence (row b * T + t)
  int H, G, D, V, DP;        // heads, q / k heads, q / k size, value size, D rounded up to 32
  int taps, C;               // convolution taps, channels (2 G D + H V)
  const void* proj;          // [B T, ldp] projections (activation type)
  int64_t ldp;
  const float* conv;         // [taps, C]
  const float* a_log;        // [H]
  const float* dt_bias;      // [H]
  const float* norm_w;       // [V]
  float qscale, eps;
  const int64_t* pos;        // position of each sequence's first new token: pos[b * pos_stride]
  int64_t pos_stride;
  const int* lens;           // [B] valid new tokens (nullable: T)
  const int* slots;          // [B] cache slots (nullable: identity)
  int nslots;
  float* state;              // [slots, H, V, DP]
  void* ring;                // [slots, taps, C] (activation type)
  float *qn, *kn;            // unit q, k: [B T, G, DP], or with nch > 0 [chunks, G, 64 DP] in fragment order
  float* vn;                 // [B T, H, V]
  float *lg, *beta;          // [B T, H] log decay, write strength
  float* o;                  // [B T, H, V]
  // 64-token chunks (csrc/hybrid/delta_chunk.hip)
  int nch;                   // chunks per sequence (0: token by token)
  float *cw, *cy, *cp;       // W [cells, 64 DP], Y [cells, 64 V rounded up to 16], P [cells, 64 64]
  float* ceg;                // [cells, 2, 64] e^G, e^(G_C - G)
  void* y;                   // [B T, ldy] mixer output before its projection (activation type)
  int64_t ldy;
};

namespace hybrid {

// the convolution inputs of a sequence's last tokens go to the ring: entry p % taps of position p
template <typename T>
__device__ __forceinline__ void ring_write(const DeltaParams& p, int b, int slot, int64_t p0, int len, int tid, int nth) {
  const int n = min(len, p.taps);
  T* ring = static_cast<T*>(p.ring) + (int64_t)slot * p.taps * p.C;
  for (int i = tid; i < n * p.C; i += nth) {
    const int t = len - n + i / p.C, c = i % p.C;
    ring[((p0 + t) % p.taps) * p.C + c] = static_cast<const T*>(p.proj)[((int64_t)b * p.T + t) * p.ldp + c];
  }
}

}  // namespace hybrid
}  // namespace nxd
