// Shared helpers of the hybrid-decoder kernels: element access for the two activation types
// (bf16 as raw uint16_t, or float), 4-wide loads, and the scalar functions of the gates.
#pragma once
#include "../common.h"

namespace nxd {
namespace hybrid {

__device__ __forceinline__ float ld(const float* p) { return *p; }
__device__ __forceinline__ float ld(const uint16_t* p) { return bf2f(*p); }
__device__ __forceinline__ void st(float* p, float v) { *p = v; }
__device__ __forceinline__ void st(uint16_t* p, float v) { *p = f2bf(v); }

__device__ __forceinline__ f32x4_t ld4(const float* p) { return *reinterpret_cast<const f32x4_t*>(p); }
__device__ __forceinline__ f32x4_t ld4(const uint16_t* p) {
  const u32x2_t v = *reinterpret_cast<const u32x2_t*>(p);
  return f32x4_t{__uint_as_float(v[0] << 16), __uint_as_float(v[0] & 0xffff0000u), __uint_as_float(v[1] << 16),
                 __uint_as_float(v[1] & 0xffff0000u)};
}
__device__ __forceinline__ void st4(float* p, const f32x4_t& v) { *reinterpret_cast<f32x4_t*>(p) = v; }
__device__ __forceinline__ void st4(uint16_t* p, const f32x4_t& v) {
  *reinterpret_cast<u32x2_t*>(p) = u32x2_t{pack2bf(v[0], v[1]), pack2bf(v[2], v[3])};
}

__device__ __forceinline__ float sigmoidf_(float x) { return 1.f / (1.f + expf(-x)); }
__device__ __forceinline__ float siluf_(float x) { return x / (1.f + expf(-x)); }
__device__ __forceinline__ float softplusf_(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

// cache slot and first position of sequence b; kept inside the cache whatever the caller's tensors hold
__device__ __forceinline__ int slot_of(const int* slots, int b, int nslots) {
  return slots ? min(max(slots[b], 0), nslots - 1) : b;
}
__device__ __forceinline__ int64_t pos_of(const int64_t* pos, int64_t stride, int b) {
  const int64_t p = pos[(int64_t)b * stride];
  return p > 0 ? p : 0;
}

}  // namespace hybrid
}  // namespace nxd
