// Parameters of the routed-expert kernels (csrc/hybrid/moe_route.hip, expert_decode.hip).
#pragma once
#include "hybrid.h"

namespace nxd {

struct RouterParams {
  int64_t M;
  int E, top, groups, keep;
  float scale;
  const float* logits;     // [M, ldl]
  int64_t ldl;
  int* index;              // [M, top]
  float* score;            // [M, top] weights by choice
  int* counts;             // [chunks, E]
  int chunks;
  int* token;              // [M top] by sorted row
  float* weight;           // [M top] by sorted row
  int* inverse;            // [M, top]
  int* offs;               // [E + 1]
};

struct GluParams {
  int64_t R;
  int F;
  const void* gu;          // [R, ldg] gate | up
  int64_t ldg;
  float limit;
  const float* weight;     // [R] with a stride (nullable)
  int64_t ldw;
  bool sigmoid;
  void* y;                 // [R, ldy]
  int64_t ldy;
};

struct ExpertRowsParams {
  const void* x;           // [X, ldx]
  int64_t ldx;
  const int* token;        // [P] (nullable: row r)
  int64_t nx;              // rows of x
  const void* w;           // [E, N, K]
  const int* offs;         // [E + 1]
  int E, N, K;
  int64_t P;
  void* y;                 // [P, N]
};

// a few tokens (expert_decode.hip)
struct LinearFewParams {
  int M, N, K;
  const uint16_t* x;       // [M, ldx]
  int64_t ldx;
  const uint16_t* w;       // [N, K]
  uint16_t* y;             // [M, ldy]
  int64_t ldy;
};

struct ExpertFewParams {
  int M, E, top, shared;   // shared: 1 with a shared expert (else 0)
  int W, F, FS;            // width, feed-forward sizes
  const uint16_t* h;       // [M, ldh]
  int64_t ldh;
  const uint16_t *router, *up, *down, *sup, *sdown;   // [E + shared, W], [E, 2 F, W], [E, W, F], [2 FS, W], [W, FS]
  float limit, slimit;
  int* index;              // [M, top]
  float* score;            // [M, top + shared]
  float* gate;             // [M] the shared expert's gate, for a caller that runs it (nullable)
  uint16_t *a, *sa;        // [M top, F], [M, FS]
  uint16_t* y;             // [M (top + shared), W]
};

namespace hybrid {

// The `top` experts of one token by one wave (E scores), largest sigmoid first, among those of the `keep`
// best groups; s [E], gsc [groups]: the wave's LDS.  chosen[j] / score[j] get expert and normalised weight.
// Every lane must call it; chosen / score are ready (for this wave) on return.
constexpr int MAX_TOP = 64;

__device__ __forceinline__ void choose_experts(const RouterParams& p, const float* z, float* s, float* gsc, int* chosen,
                                               float* score) {
  const int lane = threadIdx.x & 63, E = p.E, per = E / p.groups;
  if (lane < p.top) chosen[lane] = min(lane, E - 1), score[lane] = 0.f;   // (scores that are no numbers choose nothing)
  for (int e = lane; e < E; e += 64) s[e] = 1.f / (1.f + expf(-z[e]));
  __builtin_amdgcn_wave_barrier();
  if (p.groups > 1) {
    for (int g = lane; g < p.groups; g += 64) {
      float a = -1.f, b = -1.f;   // the two largest
      for (int i = 0; i < per; ++i) {
        const float v = s[g * per + i];
        if (v > a) b = a, a = v;
        else if (v > b) b = v;
      }
      gsc[g] = a + (per > 1 ? b : 0.f);
    }
    __builtin_amdgcn_wave_barrier();
    for (int e0 = 0; e0 < E; e0 += 64) {   // (all group scores are read before a score is struck out)
      const int e = e0 + lane, g = min(e, E - 1) / per;
      const float mine = gsc[g];
      int better = 0;
      for (int j = 0; j < p.groups; ++j) better += gsc[j] > mine || (gsc[j] == mine && j < g);
      if (e < E && better >= p.keep) s[e] = -1.f;
    }
    __builtin_amdgcn_wave_barrier();
  }
  for (int e0 = 0; e0 < E; e0 += 64) {
    const int e = e0 + lane;
    const float mine = e < E ? s[e] : -1.f;
    int better = 0;
    for (int j = 0; j < E; ++j) better += s[j] > mine || (s[j] == mine && j < e);
    if (mine >= 0.f && better < p.top) chosen[better] = e, score[better] = mine;
  }
  __builtin_amdgcn_wave_barrier();
  float sum = 0.f;
  for (int j = 0; j < p.top; ++j) sum += score[j];
  const float f = p.scale / (sum + 1e-20f);
  __builtin_amdgcn_wave_barrier();
  if (lane < p.top) score[lane] *= f;
  __builtin_amdgcn_wave_barrier();
}

// g sigmoid(1.702 g) (u + 1) of clamped gate and up
__device__ __forceinline__ float clamped_glu(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * sigmoidf_(1.702f * g) * (u + 1.f);
}

}  // namespace hybrid
}  // namespace nxd
