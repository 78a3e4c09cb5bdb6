// Preparation of attention with pooled blocks (window_attn*.hip have the attention itself):
//
//   pooled_prep : one RMS norm over all query heads of a token (in place) and one over all key heads (to a
//                 buffer of its own: the projected keys stay, they are the values), keys and values to the ring
//   pooled_mean : the means of the keys and values, as they were stored, of every block that the step's
//                 tokens complete
#include "window_attn.h"

namespace nxd {
namespace hybrid {

template <typename T, int VEC>
__device__ __forceinline__ f32x4_t load_some(const T* x) {
  if constexpr (VEC == 4) return ld4(x);
  else return f32x4_t{ld(x), 0.f, 0.f, 0.f};
}
template <typename T, int VEC>
__device__ __forceinline__ void store_some(T* x, const f32x4_t& v) {
  if constexpr (VEC == 4) st4(x, v);
  else st(x, v[0]);
}

// one workgroup a token
template <typename T, int VEC>
__global__ void __launch_bounds__(256) pooled_prep_kernel(WindowAttnParams p) {
  __shared__ float red[2][4];
  const int64_t m = blockIdx.x;
  const int b = (int)(m / p.T), t = (int)(m % p.T), tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  const int len = p.lens ? min(p.lens[b], p.T) : p.T;
  const int nq = p.H * p.D, nk = p.G * p.D, D = p.D;
  T* row = static_cast<T*>(p.buf) + m * p.ldb;
  T* kn = static_cast<T*>(const_cast<void*>(p.kbuf)) + m * p.ldk;
  if (t >= len) return;
  const int64_t ps = pos_of(p.pos, p.pos_stride, b) + t;
  const int slot = slot_of(p.slots, b, p.nslots), entry = (int)(ps % p.cap);
  const bool keep = t >= len - p.cap;   // a prompt longer than the ring: only its last entries
  float sq = 0.f, sk = 0.f;
  for (int c = tid * VEC; c < nq + nk; c += 256 * VEC) {   // VEC divides the head size
    const f32x4_t v = load_some<T, VEC>(row + c);
    const float s = v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
    if (c < nq) sq += s;
    else sk += s;
  }
  sq = sum64(sq);
  sk = sum64(sk);
  if (lane == 0) red[0][w] = sq, red[1][w] = sk;
  __syncthreads();
  sq = red[0][0] + red[0][1] + red[0][2] + red[0][3];
  sk = red[1][0] + red[1][1] + red[1][2] + red[1][3];
  const float rq = 1.f / sqrtf(sq / (float)nq + p.eps), rk = 1.f / sqrtf(sk / (float)nk + p.eps);
  for (int c = tid * VEC; c < nq + nk; c += 256 * VEC) {
    const f32x4_t v = load_some<T, VEC>(row + c);
    if (c < nq) {
      store_some<T, VEC>(row + c, v * rq * load_some<float, VEC>(p.qn_w + c));
      continue;
    }
    const int kc = c - nq;
    const f32x4_t n = v * rk * load_some<float, VEC>(p.kn_w + kc);
    store_some<T, VEC>(kn + kc, n);
    if (keep) {
      const int64_t o = (((int64_t)slot * p.G + kc / D) * p.cap + entry) * D + kc % D;
      store_some<T, VEC>(static_cast<T*>(p.kc) + o, n);
      store_some<T, VEC>(static_cast<T*>(p.vc) + o, v);
    }
  }
}

// one workgroup a block, a thread some elements of the G D of a token
template <typename T, int VEC>
__global__ void __launch_bounds__(256) pooled_mean_kernel(WindowAttnParams p) {
  const int b = blockIdx.y, nk = p.G * p.D, D = p.D, P = p.pool;
  const int len = p.lens ? min(p.lens[b], p.T) : p.T;
  if (len <= 0) return;
  const int64_t p0 = p.from_buf ? 0 : pos_of(p.pos, p.pos_stride, b);
  const int64_t blk = p0 / P + blockIdx.x;
  if ((blk + 1) * P > p0 + len || blk >= p.pcap) return;   // (not complete)
  const int slot = slot_of(p.slots, b, p.nslots);
  const float inv = 1.f / (float)P;
  for (int c = threadIdx.x * VEC; c < nk; c += 256 * VEC) {
    const int g = c / D, d = c % D;
    f32x4_t k = {0.f, 0.f, 0.f, 0.f}, v = k;
    for (int i = 0; i < P; ++i) {
      const int64_t ps = blk * P + i;
      if (p.from_buf) {
        k += load_some<T, VEC>(static_cast<const T*>(p.kbuf) + ((int64_t)b * p.T + ps) * p.ldk + c);
        v += load_some<T, VEC>(static_cast<const T*>(p.vbuf) + ((int64_t)b * p.T + ps) * p.ldv + c);
      } else {
        const int64_t o = (((int64_t)slot * p.G + g) * p.cap + ps % p.cap) * D + d;
        k += load_some<T, VEC>(static_cast<const T*>(p.kc) + o);
        v += load_some<T, VEC>(static_cast<const T*>(p.vc) + o);
      }
    }
    const int64_t o = (((int64_t)slot * p.G + g) * p.pcap + blk) * D + d;
    store_some<T, VEC>(static_cast<T*>(p.pk) + o, k * inv);
    store_some<T, VEC>(static_cast<T*>(p.pv) + o, v * inv);
  }
}

template <typename T, int VEC>
static int run_pooled_prep(const WindowAttnParams& p, hipStream_t s) {
  hipLaunchKernelGGL((pooled_prep_kernel<T, VEC>), dim3((unsigned)(p.B * p.T)), dim3(256), 0, s, p);
  // blocks that can end within T tokens, wherever they start
  hipLaunchKernelGGL((pooled_mean_kernel<T, VEC>), dim3((unsigned)(p.T / p.pool + 1), (unsigned)p.B), dim3(256), 0, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

}  // namespace hybrid

int pooled_prep_launch(bool f32, const WindowAttnParams& p, hipStream_t s) {
  using namespace hybrid;
  const bool vec = p.D % 4 == 0 && p.ldb % 4 == 0 && p.ldk % 4 == 0 && reinterpret_cast<uintptr_t>(p.buf) % 16 == 0 &&
                   reinterpret_cast<uintptr_t>(p.kbuf) % 16 == 0;
  if (f32) return vec ? run_pooled_prep<float, 4>(p, s) : run_pooled_prep<float, 1>(p, s);
  return vec ? run_pooled_prep<uint16_t, 4>(p, s) : run_pooled_prep<uint16_t, 1>(p, s);
}

}  // namespace nxd
