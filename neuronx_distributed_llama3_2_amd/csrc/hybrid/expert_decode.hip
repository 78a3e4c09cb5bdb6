// Products of a few tokens (bf16, up to 64): projections, and a whole routed feed-forward in three launches
// without sorting its pairs.
//
//   linear_few  : x w^T, up to 16 tokens
//   moe_gate    : router logits (32-bit) and the chosen experts of one token; the shared expert's gate
//   expert_few  : gate and up rows -> clamped gated activation times the pair's weight; then the down rows.
//                 The shared expert is one more expert, which every token uses
//
// Few tokens mean few rows an expert: its weights are what counts, and they are read once.  A workgroup has
// 16 weight rows (and the 16 up rows that belong to them) of one expert; each of its waves takes 128 elements
// of the reduction in turn.  Weights and tokens are read 256 contiguous bytes a row (64 at a time, as the
// operands of v_mfma_f32_16x16x32_bf16 want them, costs a quarter of the memory's rate) and change places
// in a patch of LDS that is the wave's own; 16 tokens are the B operand, and the waves' sums meet in LDS.
#include "experts.h"

namespace nxd {
namespace hybrid {

constexpr int GATE_WAVES = 16;

__global__ void __launch_bounds__(GATE_WAVES * 64) moe_gate_kernel(RouterParams r, ExpertFewParams p) {
  __shared__ float z[1025], s[1024], gsc[1024];
  __shared__ int chosen[MAX_TOP];
  __shared__ float score[MAX_TOP];
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int m = blockIdx.x, rows = p.E + (p.shared || p.gate ? 1 : 0), K = p.W;
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
  if (lane == 0 && p.shared) p.score[m * slots + p.top] = sigmoidf_(z[p.E]);
  if (lane == 0 && p.gate) p.gate[m] = sigmoidf_(z[p.E]);
}

constexpr int FEW_WAVES = 8;
constexpr int PATCH_ROW = 256 + 16, PATCH = 16 * PATCH_ROW;   // bytes

// What a lane reads: row 4 s + lane / 16 of 16 rows, s < 4, elements 8 (lane % 16) ...
struct FewRows {
  int at[4];   // offset of the row in elements; negative: none (zeros)
};

// acc[n] = 16 weight rows from w + n * second (rows K apart, of which `rows` are there) times the 16 tokens x + at[..]:
// this wave's share of the K elements (a multiple of 8).  patch: PATCH bytes of this wave
template <int NA>
__device__ __forceinline__ void few_product(const uint16_t* w, int64_t second, int rows, const uint16_t* x, const FewRows& xr, int K,
                                            char* patch, f32x4_t (&acc)[NA]) {
  constexpr int STEP = 128 * FEW_WAVES;
  const int lane = threadIdx.x & 63, lr = lane & 15, lq = lane >> 4, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
#pragma unroll
  for (int n = 0; n < NA; ++n) acc[n] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  struct Ops {
    u32x4_t w[NA][4], x[4];
  };
  const u32x4_t none = {0u, 0u, 0u, 0u};
  const uint16_t* wr[4];
#pragma unroll
  for (int s = 0; s < 4; ++s) wr[s] = w + (int64_t)min(4 * s + lq, rows - 1) * K;
  auto fetch = [&](int k0, Ops& o) {
    const int k = k0 + 8 * lr;
    const bool in = k < K;
#pragma unroll
    for (int s = 0; s < 4; ++s) {
#pragma unroll
      for (int n = 0; n < NA; ++n) o.w[n][s] = in ? __builtin_nontemporal_load(reinterpret_cast<const u32x4_t*>(wr[s] + n * second + k)) : none;
      o.x[s] = in && xr.at[s] >= 0 ? *reinterpret_cast<const u32x4_t*>(x + xr.at[s] + k) : none;
    }
  };
  auto turn = [&](u32x4_t (&v)[4]) {   // -> the lane's 8 elements 32 s + 8 lq .. of row lr
#pragma unroll
    for (int s = 0; s < 4; ++s) *reinterpret_cast<u32x4_t*>(patch + (4 * s + lq) * PATCH_ROW + lr * 16) = v[s];
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int s = 0; s < 4; ++s) v[s] = *reinterpret_cast<const u32x4_t*>(patch + lr * PATCH_ROW + 64 * s + 16 * lq);
    __builtin_amdgcn_wave_barrier();
  };
  auto use = [&](Ops& o) {
#pragma unroll
    for (int n = 0; n < NA; ++n) turn(o.w[n]);
    turn(o.x);
#pragma unroll
    for (int s = 0; s < 4; ++s)
#pragma unroll
      for (int n = 0; n < NA; ++n)
        acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, o.w[n][s]), __builtin_bit_cast(bf16x8_t, o.x[s]),
                                                         acc[n], 0, 0, 0);
  };
  Ops now, next;
  int k0 = 128 * wave;
  if (k0 < K) fetch(k0, now);
  for (; k0 < K; k0 += STEP) {
    if (k0 + STEP < K) fetch(k0 + STEP, next);
    use(now);
    now = next;
  }
}

// the waves' sums, to the first wave
template <int NA>
union FewLds {
  char patch[FEW_WAVES][PATCH];
  f32x4_t part[FEW_WAVES][NA][64];
  __device__ __forceinline__ void put(const f32x4_t (&acc)[NA]) {
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
    __syncthreads();   // (the patches' last readers are done)
#pragma unroll
    for (int n = 0; n < NA; ++n) part[w][n][lane] = acc[n];
    __syncthreads();
  }
  __device__ __forceinline__ f32x4_t get(int n) const {
    const int lane = threadIdx.x & 63;
    f32x4_t v = part[0][n][lane];
#pragma unroll
    for (int i = 1; i < FEW_WAVES; ++i) v += part[i][n][lane];
    return v;
  }
};

// y = x w^T
__global__ void __launch_bounds__(FEW_WAVES * 64) linear_few_kernel(LinearFewParams p) {
  __shared__ __attribute__((aligned(16))) FewLds<1> sums;
  const int lane = threadIdx.x & 63, lr = lane & 15, lq = lane >> 4, w = threadIdx.x >> 6, row0 = blockIdx.x * 16;
  FewRows xr;
#pragma unroll
  for (int s = 0; s < 4; ++s) xr.at[s] = 4 * s + lq < p.M ? (4 * s + lq) * (int)p.ldx : -1;
  f32x4_t acc[1];
  few_product<1>(p.w + (int64_t)row0 * p.K, 0, p.N - row0, p.x, xr, p.K, sums.patch[w], acc);
  sums.put(acc);
  const int n = row0 + 4 * lq;
  if (w > 0 || lr >= p.M) return;
  const f32x4_t v = sums.get(0);
  uint16_t* y = p.y + (int64_t)lr * p.ldy + n;
  if (n + 4 <= p.N && p.ldy % 4 == 0) {
    st4(y, v);
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (n + i < p.N) st(y + i, v[i]);
  }
}

// UP: a[pair] = activation of h; else y[slot] = down rows times a[pair]
template <bool UP>
__global__ void __launch_bounds__(FEW_WAVES * 64) expert_few_kernel(ExpertFewParams p) {
  constexpr int NA = UP ? 2 : 1;
  __shared__ int list[64];   // the expert's pairs m * top + j
  __shared__ __attribute__((aligned(16))) FewLds<NA> sums;
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
  cnt = min(cnt, p.M);
  __syncthreads();
  const int N = UP ? (is_shared ? p.FS : p.F) : p.W, K = UP ? p.W : (is_shared ? p.FS : p.F);
  const uint16_t* wm = UP ? (is_shared ? p.sup : p.up + (int64_t)e * 2 * p.F * K) : (is_shared ? p.sdown : p.down + (int64_t)e * p.W * K);
  const uint16_t* x = UP ? p.h : (is_shared ? p.sa : p.a);
  for (int r0 = 0; r0 < cnt; r0 += 16) {   // (more than 16 rows of an expert: its weights again, from the cache)
    FewRows xr;
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const int r = r0 + 4 * s + lq, pr = r < cnt ? list[r] : -1;
      xr.at[s] = pr < 0 ? -1 : (UP ? pr / top * (int)p.ldh : (is_shared ? pr / top * p.FS : pr * p.F));
    }
    f32x4_t acc[NA];
    if (r0 > 0) __syncthreads();   // (the last tile's sums have been read)
    few_product<NA>(wm + (int64_t)row0 * K, (int64_t)N * K, N - row0, x, xr, K, sums.patch[w], acc);
    sums.put(acc);
    if (w > 0 || r0 + lr >= cnt || row0 + 4 * lq >= N) continue;   // rows row0 + 4 lq .. + 3 of token lr
    const int pr = list[r0 + lr], m = pr / top, slot = m * slots + (is_shared ? top : pr % top);
    if constexpr (UP) {
      const f32x4_t g = sums.get(0), u = sums.get(1);
      const float weight = p.score[slot], limit = is_shared ? p.slimit : p.limit;
      f32x4_t o;
#pragma unroll
      for (int i = 0; i < 4; ++i) o[i] = clamped_glu(g[i], u[i], limit) * weight;
      st4((is_shared ? p.sa + (int64_t)m * p.FS : p.a + (int64_t)pr * p.F) + row0 + 4 * lq, o);
    } else {
      st4(p.y + (int64_t)slot * p.W + row0 + 4 * lq, sums.get(0));
    }
  }
}

template <bool UP>
static void launch_few(const ExpertFewParams& p, hipStream_t s) {
  const int q = p.M * p.top < p.E ? p.M * p.top : p.E;
  const int per_shared = p.shared ? ceil_div(UP ? p.FS : p.W, 16) : 0, per = ceil_div(UP ? p.F : p.W, 16);
  hipLaunchKernelGGL((expert_few_kernel<UP>), dim3((unsigned)(per_shared + q * per)), dim3(FEW_WAVES * 64), 0, s, p);
}

}  // namespace hybrid

int experts_few_launch(const RouterParams& r, const ExpertFewParams& p, hipStream_t s) {
  if (p.M > 64 || p.top > hybrid::MAX_TOP || p.E > 1024) return -1;
  hipLaunchKernelGGL(hybrid::moe_gate_kernel, dim3((unsigned)p.M), dim3(hybrid::GATE_WAVES * 64), 0, s, r, p);
  hybrid::launch_few<true>(p, s);
  hybrid::launch_few<false>(p, s);
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

int linear_few_launch(const LinearFewParams& p, hipStream_t s) {
  if (p.M < 1 || p.M > 16 || p.K % 8) return -1;
  hipLaunchKernelGGL(hybrid::linear_few_kernel, dim3((unsigned)ceil_div(p.N, 16)), dim3(hybrid::FEW_WAVES * 64), 0, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

}  // namespace nxd
