// The step between two layers whose sublayers read one fp32 residual side by side:
//
//   x <- x (or an embedding row) + outputs of the last layer (up to two rows, and k rows of expert outputs
//        found through `inverse`, or in order)
//   h_n = x / sqrt(mean over each of `groups` equal parts of x^2 + eps) * w_n      (one or two weights)
//
// One workgroup a row, the row in registers, 4 elements a lane and step (1 for sizes that are no multiple).
#include "group_norm.h"

namespace nxd {
namespace hybrid {

template <int VEC>
struct Vec {
  float v[VEC];
};
template <int VEC, typename T>
__device__ __forceinline__ Vec<VEC> load(const T* p) {
  Vec<VEC> r;
  if constexpr (VEC == 4) {
    const f32x4_t t = ld4(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) r.v[i] = t[i];
  } else {
    r.v[0] = ld(p);
  }
  return r;
}
template <int VEC, typename T>
__device__ __forceinline__ void store(T* p, const Vec<VEC>& x) {
  if constexpr (VEC == 4) st4(p, f32x4_t{x.v[0], x.v[1], x.v[2], x.v[3]});
  else st(p, x.v[0]);
}

template <typename T, int VEC, int NV>
__global__ void __launch_bounds__(256) residual_norms_kernel(GroupNormParams p) {
  extern __shared__ float sums[];   // [W / VEC] (groups > 1), then [groups]
  __shared__ float red[16];
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, W = p.W;
  const int64_t r = blockIdx.x, m = p.rows ? min(max(p.rows[r], (int64_t)0), p.M - 1) : r;
  const T* e = nullptr;
  bool zero = false;
  if (p.embed) {
    const int64_t id = p.ids[m];
    zero = id < 0 || id >= p.vocab;
    e = static_cast<const T*>(p.embed) + (zero ? 0 : id) * W;
  }
  float* xr = p.x + m * W;
  Vec<VEC> x[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * 256 + tid) * VEC;
    if (c < W) {
      x[i] = e ? load<VEC>(e + c) : load<VEC>(xr + c);
      if (zero) x[i] = Vec<VEC>{};
    } else {
      x[i] = Vec<VEC>{};
    }
  }
#pragma unroll
  for (int a = 0; a < 2; ++a) {
    if (!p.add[a]) continue;
    const T* s = static_cast<const T*>(p.add[a]) + m * p.ld_add[a];
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * 256 + tid) * VEC;
      if (c >= W) continue;
      const Vec<VEC> t = load<VEC>(s + c);
#pragma unroll
      for (int j = 0; j < VEC; ++j) x[i].v[j] += t.v[j];
    }
  }
  if (p.pairs) {
    for (int k = 0; k < p.k; ++k) {
      const int row = p.inverse ? min(max(p.inverse[m * p.k + k], 0), p.npairs - 1) : (int)(m * p.k + k);
      const T* s = static_cast<const T*>(p.pairs) + (int64_t)row * W;
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int c = (i * 256 + tid) * VEC;
        if (c >= W) continue;
        const Vec<VEC> t = load<VEC>(s + c);
#pragma unroll
        for (int j = 0; j < VEC; ++j) x[i].v[j] += t.v[j];
      }
    }
  }
  if (p.store) {
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * 256 + tid) * VEC;
      if (c < W) store<VEC>(xr + c, x[i]);
    }
  }
  if (!p.h[0]) return;
  const int part = W / p.groups;
  float rs = 0.f;
  float* gs = sums + W / VEC;
  if (p.groups == 1) {
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
      for (int j = 0; j < VEC; ++j) ss += x[i].v[j] * x[i].v[j];
    rs = 1.f / sqrtf(block_sum(ss, red) / (float)W + p.eps);
  } else {
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = i * 256 + tid;
      float ss = 0.f;
#pragma unroll
      for (int j = 0; j < VEC; ++j) ss += x[i].v[j] * x[i].v[j];
      if (c * VEC < W) sums[c] = ss;
    }
    __syncthreads();
    const int n = part / VEC;   // pieces of a group: VEC divides the part
    for (int g = wid; g < p.groups; g += 4) {
      float ss = 0.f;
      for (int i = lane; i < n; i += 64) ss += sums[g * n + i];
      ss = sum64(ss);
      if (lane == 0) gs[g] = 1.f / sqrtf(ss / (float)part + p.eps);
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * 256 + tid) * VEC;
    if (c >= W) continue;
    const float f = p.groups == 1 ? rs : gs[c / part];
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      if (!p.h[n]) continue;
      const Vec<VEC> w = load<VEC>(p.w[n] + c);
      Vec<VEC> y;
#pragma unroll
      for (int j = 0; j < VEC; ++j) y.v[j] = x[i].v[j] * f * w.v[j];
      store<VEC>(static_cast<T*>(p.h[n]) + r * p.ldh + c, y);
    }
  }
}

template <typename T, int VEC, int NV>
static int run_norms(const GroupNormParams& p, hipStream_t s) {
  const size_t lds = p.groups > 1 ? (size_t)(p.W / VEC + p.groups) * 4 : 0;
  static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(&residual_norms_kernel<T, VEC, NV>),
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, 144 * 1024);
  if (attr != hipSuccess) return 2;
  hipLaunchKernelGGL((residual_norms_kernel<T, VEC, NV>), dim3((unsigned)p.R), dim3(256), lds, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

template <typename T>
static int by_width(const GroupNormParams& p, bool vec, hipStream_t s) {
  if (vec) {
    if (p.W <= 1024) return run_norms<T, 4, 1>(p, s);
    if (p.W <= 2048) return run_norms<T, 4, 2>(p, s);
    if (p.W <= 4096) return run_norms<T, 4, 4>(p, s);
    if (p.W <= 8192) return run_norms<T, 4, 8>(p, s);
    return run_norms<T, 4, 16>(p, s);
  }
  if (p.W <= 1024) return run_norms<T, 1, 4>(p, s);
  if (p.W <= 4096) return run_norms<T, 1, 16>(p, s);
  return run_norms<T, 1, 64>(p, s);
}

}  // namespace hybrid

int residual_norms_launch(bool f32, const GroupNormParams& p, bool vec, hipStream_t s) {
  return f32 ? hybrid::by_width<float>(p, vec, s) : hybrid::by_width<uint16_t>(p, vec, s);
}

}  // namespace nxd
