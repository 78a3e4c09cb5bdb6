// Router of a mixture of experts without a host sync:
//
//   moe_choose : scores, groups, the chosen experts and their weights of a chunk of tokens (a wave a token),
//                and the chunk's count of every expert
//   moe_scan   : where every chunk's pairs of every expert start when pairs are sorted by expert
//   moe_place  : where every (token, choice) pair goes (stable)
//
// and what runs around the experts' matrix products: the gather of token rows and the clamped gated
// activation with the pair's weight.
#include "experts.h"

namespace nxd {
namespace hybrid {

constexpr int ROUTE_TOKENS = 32;   // tokens of a chunk
constexpr int ROUTE_WAVES = 8;

__global__ void __launch_bounds__(ROUTE_WAVES * 64) moe_choose_kernel(RouterParams p) {
  extern __shared__ __attribute__((aligned(16))) float smem[];   // per wave: E scores, `groups` sums; then E counts
  __shared__ int chosen[ROUTE_WAVES][MAX_TOP];
  __shared__ float score[ROUTE_WAVES][MAX_TOP];
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, E = p.E;
  float* s = smem + w * (E + p.groups);
  int* count = reinterpret_cast<int*>(smem + ROUTE_WAVES * (E + p.groups));
  for (int e = tid; e < E; e += ROUTE_WAVES * 64) count[e] = 0;
  __syncthreads();
  for (int t = w; t < ROUTE_TOKENS; t += ROUTE_WAVES) {
    const int64_t m = (int64_t)blockIdx.x * ROUTE_TOKENS + t;
    if (m >= p.M) break;
    choose_experts(p, p.logits + m * p.ldl, s, s + E, chosen[w], score[w]);
    if (lane < p.top) {
      p.index[m * p.top + lane] = chosen[w][lane];
      p.score[m * p.top + lane] = score[w][lane];
      atomicAdd(count + chosen[w][lane], 1);
    }
    __builtin_amdgcn_wave_barrier();
  }
  __syncthreads();
  for (int e = tid; e < E; e += ROUTE_WAVES * 64) p.counts[(int64_t)blockIdx.x * E + e] = count[e];
}

// counts[chunk][e] -> the chunk's first row of expert e; offs.  One workgroup, a wave an expert at a time
__global__ void __launch_bounds__(1024) moe_scan_kernel(RouterParams p) {
  extern __shared__ int total[];   // [E + 1]
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, E = p.E;
  for (int e = w; e < E; e += 16) {
    int run = 0;
    for (int c0 = 0; c0 < p.chunks; c0 += 64) {
      const int c = c0 + lane, n = c < p.chunks ? p.counts[(int64_t)c * E + e] : 0;
      int x = n;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const int y = __shfl_up(x, o, 64);
        if (lane >= o) x += y;
      }
      if (c < p.chunks) p.counts[(int64_t)c * E + e] = run + x - n;
      run += __shfl(x, 63, 64);
    }
    if (lane == 0) total[e] = run;
  }
  __syncthreads();
  if (w == 0) {
    int run = 0;
    for (int e0 = 0; e0 < E; e0 += 64) {
      const int e = e0 + lane, n = e < E ? total[e] : 0;
      int x = n;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const int y = __shfl_up(x, o, 64);
        if (lane >= o) x += y;
      }
      if (e < E) p.offs[e] = run + x - n;
      run += __shfl(x, 63, 64);
    }
    if (lane == 0) p.offs[E] = run;
  }
}

// a thread a (token, choice) pair of the chunk
__global__ void __launch_bounds__(256) moe_place_kernel(RouterParams p) {
  extern __shared__ __attribute__((aligned(16))) int ex[];   // the chunk's experts
  const int tid = threadIdx.x, ch = blockIdx.x, E = p.E, top = p.top;
  const int64_t i0 = (int64_t)ch * ROUTE_TOKENS * top;
  const int n = (int)min((int64_t)ROUTE_TOKENS * top, p.M * top - i0);
  for (int i = tid; i < n; i += 256) ex[i] = p.index[i0 + i];
  __syncthreads();
  for (int i = tid; i < n; i += 256) {
    const int e = ex[i];
    int at = p.offs[e] + p.counts[(int64_t)ch * E + e];
    for (int j = 0; j < i; ++j) at += ex[j] == e;
    p.token[at] = (int)((i0 + i) / top);
    p.weight[at] = p.score[i0 + i];
    p.inverse[i0 + i] = at;
  }
}

template <typename T, int VEC>
__global__ void __launch_bounds__(256) clamped_glu_kernel(GluParams p) {
  const int per = p.F / VEC;
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= p.R * per) return;
  const int64_t r = i / per;
  const int c = (int)(i % per) * VEC;
  const T* g = static_cast<const T*>(p.gu) + r * p.ldg + c;
  T* y = static_cast<T*>(p.y) + r * p.ldy + c;
  float w = p.weight ? p.weight[r * p.ldw] : 1.f;
  if (p.sigmoid) w = sigmoidf_(w);
  if constexpr (VEC == 4) {
    const f32x4_t a = ld4(g), b = ld4(g + p.F);
    f32x4_t o;
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] = clamped_glu(a[j], b[j], p.limit) * w;
    st4(y, o);
  } else {
    st(y, clamped_glu(ld(g), ld(g + p.F), p.limit) * w);
  }
}

__global__ void __launch_bounds__(256) gather_rows_kernel(const u32x4_t* x, const int* token, u32x4_t* y, int64_t nx, int64_t P, int n) {
  const int64_t r = blockIdx.x;
  const int64_t t = min(max((int64_t)token[r], (int64_t)0), nx - 1);
  for (int i = threadIdx.x; i < n; i += 256) y[r * n + i] = x[t * n + i];
}

// y[r] = x[token[r]] w[e]^T for a row of expert e: any sizes, a workgroup a row, a wave an output
template <typename T>
__global__ void __launch_bounds__(256) expert_rows_kernel(ExpertRowsParams p) {
  extern __shared__ float xs[];
  const int64_t r = blockIdx.x;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  int lo = 0, hi = p.E;   // the expert whose rows contain r: offs[lo] <= r < offs[lo + 1]
  while (hi - lo > 1) {
    const int mid = (lo + hi) / 2;
    if (p.offs[mid] <= r) lo = mid;
    else hi = mid;
  }
  const int64_t src = p.token ? min(max((int64_t)p.token[r], (int64_t)0), p.nx - 1) : r;
  const T* x = static_cast<const T*>(p.x) + src * p.ldx;
  for (int k = tid; k < p.K; k += 256) xs[k] = ld(x + k);
  __syncthreads();
  for (int n = w; n < p.N; n += 4) {
    const T* wr = static_cast<const T*>(p.w) + ((int64_t)lo * p.N + n) * p.K;
    float a = 0.f;
    for (int k = lane; k < p.K; k += 64) a += xs[k] * ld(wr + k);
    a = sum64(a);
    if (lane == 0) st(static_cast<T*>(p.y) + r * p.N + n, a);
  }
}

}  // namespace hybrid

int moe_route_chunk() { return hybrid::ROUTE_TOKENS; }

int moe_route_launch(const RouterParams& p, hipStream_t s) {
  using namespace hybrid;
  if (p.top > MAX_TOP || p.E > 1024) return -1;
  const size_t lds = (size_t)(ROUTE_WAVES * (p.E + p.groups) + p.E) * 4;
  static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(&moe_choose_kernel),
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024);
  if (attr != hipSuccess) return 2;
  hipLaunchKernelGGL(moe_choose_kernel, dim3((unsigned)p.chunks), dim3(ROUTE_WAVES * 64), lds, s, p);
  hipLaunchKernelGGL(moe_scan_kernel, dim3(1), dim3(1024), (size_t)(p.E + 1) * 4, s, p);
  hipLaunchKernelGGL(moe_place_kernel, dim3((unsigned)p.chunks), dim3(256), (size_t)ROUTE_TOKENS * p.top * 4, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

int clamped_glu_launch(bool f32, const GluParams& p, bool vec, hipStream_t s) {
  using namespace hybrid;
  const dim3 grid((unsigned)ceil_div64(p.R * (p.F / (vec ? 4 : 1)), 256)), block(256);
  if (f32 && vec) hipLaunchKernelGGL((clamped_glu_kernel<float, 4>), grid, block, 0, s, p);
  else if (f32) hipLaunchKernelGGL((clamped_glu_kernel<float, 1>), grid, block, 0, s, p);
  else if (vec) hipLaunchKernelGGL((clamped_glu_kernel<uint16_t, 4>), grid, block, 0, s, p);
  else hipLaunchKernelGGL((clamped_glu_kernel<uint16_t, 1>), grid, block, 0, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

int gather_rows_launch(const void* x, const int* token, void* y, int64_t nx, int64_t P, int64_t row_bytes, hipStream_t s) {
  hipLaunchKernelGGL(hybrid::gather_rows_kernel, dim3((unsigned)P), dim3(256), 0, s, static_cast<const u32x4_t*>(x), token,
                     static_cast<u32x4_t*>(y), nx, P, (int)(row_bytes / 16));
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

int expert_rows_launch(bool f32, const ExpertRowsParams& p, hipStream_t s) {
  using namespace hybrid;
  const size_t lds = (size_t)p.K * 4;
  if (lds > 160 * 1024) return -1;
  static const hipError_t a1 = hipFuncSetAttribute(reinterpret_cast<const void*>(&expert_rows_kernel<float>),
                                                   hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
  static const hipError_t a2 = hipFuncSetAttribute(reinterpret_cast<const void*>(&expert_rows_kernel<uint16_t>),
                                                   hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
  if (a1 != hipSuccess || a2 != hipSuccess) return 2;
  if (f32) hipLaunchKernelGGL((expert_rows_kernel<float>), dim3((unsigned)p.P), dim3(256), lds, s, p);
  else hipLaunchKernelGGL((expert_rows_kernel<uint16_t>), dim3((unsigned)p.P), dim3(256), lds, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

}  // namespace nxd
