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
// two neighbouring elements (aligned to the pair)
__device__ __forceinline__ void ld2(const float* p, float& a, float& b) {
  const float2 v = *reinterpret_cast<const float2*>(p);
  a = v.x;
  b = v.y;
}
__device__ __forceinline__ void ld2(const uint16_t* p, float& a, float& b) {
  const uint32_t v = *reinterpret_cast<const uint32_t*>(p);
  a = __uint_as_float(v << 16);
  b = __uint_as_float(v & 0xffff0000u);
}
__device__ __forceinline__ void st4(float* p, const f32x4_t& v) { *reinterpret_cast<f32x4_t*>(p) = v; }
__device__ __forceinline__ void st4(uint16_t* p, const f32x4_t& v) {
  *reinterpret_cast<u32x2_t*>(p) = u32x2_t{pack2bf(v[0], v[1]), pack2bf(v[2], v[3])};
}

// 1 / (1 + e^-x) from the hardware's exp2 and reciprocal (1 ulp each)
__device__ __forceinline__ float sigmoidf_(float x) {
  return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * x));
}
__device__ __forceinline__ float siluf_(float x) { return x * sigmoidf_(x); }

// Workgroup barrier for data handed over in LDS only: global loads stay in flight across it
// (__syncthreads waits for all of them, which makes every prefetch useless)
__device__ __forceinline__ void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}

// sum over the wave's 64 lanes by DPP moves and the half swaps (no LDS crossbar)
template <int CTRL>
__device__ __forceinline__ float dpp_add(float x) {
  return x + __uint_as_float(__builtin_amdgcn_update_dpp(0, __float_as_uint(x), CTRL, 0xf, 0xf, true));
}
__device__ __forceinline__ float sum16(float x) {   // each row of 16 lanes
  x = dpp_add<0xB1>(x);    // quad_perm 1 0 3 2
  x = dpp_add<0x4E>(x);    // quad_perm 2 3 0 1
  x = dpp_add<0x141>(x);   // row_half_mirror
  return dpp_add<0x140>(x);  // row_mirror
}
__device__ __forceinline__ float sum64(float x) {
  x = sum16(x);
  auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(x), __float_as_uint(x), false, false);
  x = __uint_as_float(a[0]) + __uint_as_float(a[1]);
  auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
  return __uint_as_float(b[0]) + __uint_as_float(b[1]);
}
template <int CTRL>
__device__ __forceinline__ float dpp_max(float x) {
  return fmaxf(x, __uint_as_float(__builtin_amdgcn_update_dpp(0, __float_as_uint(x), CTRL, 0xf, 0xf, true)));
}
__device__ __forceinline__ float max64(float x) {
  x = dpp_max<0x140>(dpp_max<0x141>(dpp_max<0x4E>(dpp_max<0xB1>(x))));
  auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(x), __float_as_uint(x), false, false);
  x = fmaxf(__uint_as_float(a[0]), __uint_as_float(a[1]));
  auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
  return fmaxf(__uint_as_float(b[0]), __uint_as_float(b[1]));
}
template <int N>
__device__ __forceinline__ float sum_lanes(float x) {   // each aligned group of N = 4, 8, 16, 32 or 64 lanes
  x = dpp_add<0xB1>(x);
  x = dpp_add<0x4E>(x);
  if (N >= 8) x = dpp_add<0x141>(x);
  if (N >= 16) x = dpp_add<0x140>(x);
  if (N >= 32) {
    auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(x), __float_as_uint(x), false, false);
    x = __uint_as_float(a[0]) + __uint_as_float(a[1]);
  }
  if (N >= 64) {
    auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
    x = __uint_as_float(b[0]) + __uint_as_float(b[1]);
  }
  return x;
}
__device__ __forceinline__ float sum8(float x) {   // each aligned group of 8 lanes
  x = dpp_add<0xB1>(x);
  x = dpp_add<0x4E>(x);
  return dpp_add<0x141>(x);
}
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
