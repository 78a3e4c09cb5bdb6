// Routed experts and the shared expert for a few tokens (bf16, up to 64): three launches, nothing is sorted.
//
//   moe_gate    : router logits (32-bit) and the chosen experts of one token; the shared expert's gate
//   expert_few  : gate and up rows -> clamped gated activation times the pair's weight; then the down rows.
//                 The shared expert is one more expert, which every token uses
//
// Few tokens mean few rows an expert: its weights are what counts, and they are read once.  A workgroup has
// 16 weight rows (and the 16 up rows that belong to them) of one expert; its four waves take every fourth
// 128 elements of the reduction, weights straight from memory into the A operand of
// v_mfma_f32_16x16x32_bf16, up to NT tiles of 16 tokens as B; the sums meet in LDS.
#include "experts.h"

namespace nxd {
namespace hybrid {

constexpr int GATE_WAVES = 16;

__global__ void __launch_bounds__(GATE_WAVES * 64) moe_gate_kernel(RouterParams r, ExpertFewParams p) {
  __shared__ float z[1025], s[1024], gsc[1024];
  __shared__ int chosen[MAX_TOP];
  __shared__ float score[MAX_TOP];
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int m = blockIdx.x, rows = p.E + p.shared, K = p.W;
  const uint16_t* x = p.h + (int64_t)m * p.ldh;
  for (int r0 = w; r0 < rows; r0 += 4 * GATE_WAVES) {   // four rows at a time
    const uint16_t* wr[4];
    float a[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < 4; ++j) wr[j] = p.router + (int64_t)min(r0 + j * GATE_WAVES, rows - 1) * K;
#pragma unroll 4
    for (int k = lane * 8; k < K; k += 512) {
      const u32x4_t xv = *reinterpret_cast<const u32x4_t*>(x + k);
#pragma unroll
      for (int j = 0; j < 4; ++j) a[j] = dot8_bf16(xv, *reinterpret_cast<const u32x4_t*>(wr[j] + k), a[j]);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      a[j] = sum64(a[j]);
      if (lane == 0 && r0 + j * GATE_WAVES < rows) z[r0 + j * GATE_WAVES] = a[j];
    }
  }
  __syncthreads();
  if (w != 0) return;
  choose_experts(r, z, s, gsc, chosen, score);
  const int slots = p.top + p.shared;
  if (lane < p.top) {
    p.index[m * p.top + lane] = chosen[lane];
    p.score[m * slots + lane] = score[lane];
  }
  if (p.shared && lane == 0) p.score[m * slots + p.top] = sigmoidf_(z[p.E]);
}

// UP: a[pair] = activation of h; else y[slot] = down rows times a[pair]
template <int NT, bool UP>
__global__ void __launch_bounds__(256) expert_few_kernel(ExpertFewParams p) {
  constexpr int NA = UP ? 2 : 1;
  __shared__ int list[64];                                             // the expert's pairs m * top + j
  __shared__ __attribute__((aligned(16))) f32x4_t part[4][NA * NT][64];
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lq = lane >> 4;
  const int top = p.top, slots = top + p.shared, P = p.M * top;
  const int per_shared = p.shared ? ceil_div(UP ? p.FS : p.W, 16) : 0, per = ceil_div(UP ? p.F : p.W, 16);
  int blk = blockIdx.x;
  const bool is_shared = blk < per_shared;
  if (!is_shared) blk -= per_shared;
  const int q = is_shared ? 0 : blk / per, row0 = (is_shared ? blk : blk % per) * 16;
  int e = q, cnt;
  if (is_shared) {
    cnt = p.M;
    if (tid < p.M) list[tid] = tid * top;   // (its token)
  } else {
    if (P < p.E) {   // one block of workgroups a pair: the first pair of an expert takes all of them
      e = p.index[q];
      for (int i = 0; i < q; ++i)
        if (p.index[i] == e) return;
    }
    cnt = 0;
    for (int i0 = 0; i0 < P; i0 += 64) {   // (every wave counts, the first one writes)
      const bool mine = i0 + lane < P && p.index[min(i0 + lane, P - 1)] == e;
      const uint64_t all = __ballot(mine);
      const int at = cnt + __popcll(all & ((1ull << lane) - 1));
      if (mine && w == 0 && at < 64) list[at] = i0 + lane;
      cnt += __popcll(all);
    }
    if (cnt == 0) return;
    e = min(max(e, 0), p.E - 1);
  }
  cnt = min(cnt, 16 * NT);
  __syncthreads();
  const int N = UP ? (is_shared ? p.FS : p.F) : p.W, K = UP ? p.W : (is_shared ? p.FS : p.F);
  const uint16_t* wm = UP ? (is_shared ? p.sup : p.up + (int64_t)e * 2 * p.F * K) : (is_shared ? p.sdown : p.down + (int64_t)e * p.W * K);
  const uint16_t* wr = wm + (int64_t)min(row0 + lr, N - 1) * K;
  const uint16_t* xr[NT];
  int pair[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    pair[t] = t * 16 + lr < cnt ? list[t * 16 + lr] : -1;
    const int pr = max(pair[t], 0);
    xr[t] = UP ? p.h + (int64_t)(pr / top) * p.ldh : (is_shared ? p.sa + (int64_t)(pr / top) * p.FS : p.a + (int64_t)pr * p.F);
  }
  f32x4_t acc[NA][NT];
#pragma unroll
  for (int n = 0; n < NA; ++n)
#pragma unroll
    for (int t = 0; t < NT; ++t) acc[n][t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  struct Ops {
    u32x4_t w[NA][4], x[NT][4];
  };
  const u32x4_t none = {0u, 0u, 0u, 0u};
  auto fetch = [&](int k0, Ops& o) {
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const int k = k0 + 32 * s + 8 * lq;
      const bool in = k < K;   // K is a multiple of 8
#pragma unroll
      for (int n = 0; n < NA; ++n) o.w[n][s] = in ? __builtin_nontemporal_load(reinterpret_cast<const u32x4_t*>(wr + (int64_t)n * N * K + k)) : none;
#pragma unroll
      for (int t = 0; t < NT; ++t) o.x[t][s] = in && pair[t] >= 0 ? *reinterpret_cast<const u32x4_t*>(xr[t] + k) : none;
    }
  };
  auto use = [&](const Ops& o) {
#pragma unroll
    for (int s = 0; s < 4; ++s)
#pragma unroll
      for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int n = 0; n < NA; ++n)
          acc[n][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, o.w[n][s]),
                                                              __builtin_bit_cast(bf16x8_t, o.x[t][s]), acc[n][t], 0, 0, 0);
  };
  Ops now, next;
  int k0 = 128 * w;
  if (k0 < K) fetch(k0, now);
  for (; k0 < K; k0 += 512) {
    if (k0 + 512 < K) fetch(k0 + 512, next);
    use(now);
    now = next;
  }
#pragma unroll
  for (int n = 0; n < NA; ++n)
#pragma unroll
    for (int t = 0; t < NT; ++t) part[w][n * NT + t][lane] = acc[n][t];
  __syncthreads();
  const int t = w;   // a wave finishes a tile: rows row0 + 4 lq .. + 3 of token lr
  if (t >= NT || t * 16 + lr >= cnt || row0 + 4 * lq >= N) return;
  f32x4_t v[NA];
#pragma unroll
  for (int n = 0; n < NA; ++n) v[n] = part[0][n * NT + t][lane] + part[1][n * NT + t][lane] + part[2][n * NT + t][lane] + part[3][n * NT + t][lane];
  const int pr = list[t * 16 + lr], m = pr / top, slot = m * slots + (is_shared ? top : pr % top);
  if constexpr (UP) {
    const float weight = p.score[slot], limit = is_shared ? p.slimit : p.limit;
    f32x4_t o;
#pragma unroll
    for (int i = 0; i < 4; ++i) o[i] = clamped_glu(v[0][i], v[NA - 1][i], limit) * weight;
    st4((is_shared ? p.sa + (int64_t)m * p.FS : p.a + (int64_t)pr * p.F) + row0 + 4 * lq, o);
  } else {
    st4(p.y + (int64_t)slot * p.W + row0 + 4 * lq, v[0]);
  }
}

template <bool UP>
static void launch_few(const ExpertFewParams& p, hipStream_t s) {
  const int q = p.M * p.top < p.E ? p.M * p.top : p.E;
  const int per_shared = p.shared ? ceil_div(UP ? p.FS : p.W, 16) : 0, per = ceil_div(UP ? p.F : p.W, 16);
  const dim3 grid((unsigned)(per_shared + q * per)), block(256);
  if (p.M <= 16) hipLaunchKernelGGL((expert_few_kernel<1, UP>), grid, block, 0, s, p);
  else if (p.M <= 32) hipLaunchKernelGGL((expert_few_kernel<2, UP>), grid, block, 0, s, p);
  else hipLaunchKernelGGL((expert_few_kernel<4, UP>), grid, block, 0, s, p);
}

}  // namespace hybrid

int experts_few_launch(const RouterParams& r, const ExpertFewParams& p, hipStream_t s) {
  if (p.M > 64 || p.top > hybrid::MAX_TOP || p.E > 1024) return -1;
  hipLaunchKernelGGL(hybrid::moe_gate_kernel, dim3((unsigned)p.M), dim3(hybrid::GATE_WAVES * 64), 0, s, r, p);
  hybrid::launch_few<true>(p, s);
  hybrid::launch_few<false>(p, s);
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

}  // namespace nxd
