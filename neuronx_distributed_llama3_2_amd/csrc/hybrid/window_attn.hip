// Causal attention with a sliding window, score soft-capping and one or two maps per head
// (differential attention), over a per-layer ring cache; optionally with one key and value for each block
// of tokens before the window (one map, pooled_attn.hip).
//
//   attn_prep   : bias, per-head RMS norm of q / k, rotary turn of the pairs (2i, 2i + 1) of the first
//                 `rot` dimensions, in place in the projection buffer; k and v also to the cache
//   attn_row    : one wave per (token, head), keys across lanes -- any size, fp32 or bf16, keys of the
//                 buffer (prompt) or of the cache (any number of new tokens)
//   attn_prompt : bf16 prompts on the matrix cores (window_attn_prompt.h)
//   attn_decode : one new token per sequence, preparation included (window_attn_decode.hip)
//
// A key at position p lives in entry p % cap of the cache, so a windowed layer keeps about a window of
// keys however long the sequence is.  Scores and weights are fp32.
#include "window_attn.h"

namespace nxd {
namespace hybrid {

template <typename T>
__global__ void __launch_bounds__(256) attn_prep_kernel(WindowAttnParams p) {
  const int64_t m = blockIdx.x;
  const int b = (int)(m / p.T), t = (int)(m % p.T);
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int len = p.lens ? min(p.lens[b], p.T) : p.T;
  if (t >= len) return;
  const int64_t ps = pos_of(p.pos, p.pos_stride, b) + t;
  const int64_t pt = ps < p.max_pos ? ps : p.max_pos - 1;
  const int slot = slot_of(p.slots, b, p.nslots);
  const int entry = (int)(ps % p.cap);
  const bool keep = t >= len - p.cap;   // a prompt longer than the ring: only its last entries
  T* row = static_cast<T*>(p.buf) + m * p.ldb;
  const int nq = p.H * p.maps, nk = p.G * p.maps, D = p.D, V = p.V, half = p.rot / 2;
  for (int hd = wid; hd < nq + nk + p.G; hd += 4) {
    if (hd < nq + nk) {
      T* x = row + hd * D;
      const float* nw = hd < nq ? p.qn_w : p.kn_w;
      float u[2], w[2], ss = 0.f;
#pragma unroll
      for (int i = 0; i < 2; ++i) {   // pair lane + 64 i
        const int d = 2 * (lane + 64 * i);
        u[i] = d < D ? ld(x + d) + (p.bias ? p.bias[hd * D + d] : 0.f) : 0.f;
        w[i] = d + 1 < D ? ld(x + d + 1) + (p.bias ? p.bias[hd * D + d + 1] : 0.f) : 0.f;
        ss += u[i] * u[i] + w[i] * w[i];
      }
      const float r = nw ? 1.f / sqrtf(wave_sum(ss) / (float)D + p.eps) : 1.f;
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const int pr = lane + 64 * i, d = 2 * pr;
        if (d >= D) continue;
        float a = u[i] * r, c = w[i] * r;
        if (nw) {
          a *= nw[d];
          if (d + 1 < D) c *= nw[d + 1];
        }
        if (pr < half) {
          const float cs = p.cos_t[pt * half + pr], sn = p.sin_t[pt * half + pr];
          const float a2 = a * cs - c * sn;
          c = c * cs + a * sn;
          a = a2;
        }
        st(x + d, a);
        if (d + 1 < D) st(x + d + 1, c);
        if (hd >= nq && keep) {
          T* k = static_cast<T*>(p.kc) + (((int64_t)slot * nk + (hd - nq)) * p.cap + entry) * D;
          st(k + d, a);
          if (d + 1 < D) st(k + d + 1, c);
        }
      }
    } else {
      const int g = hd - nq - nk, c0 = (nq + nk) * D + g * V;
      T* v = static_cast<T*>(p.vc) + (((int64_t)slot * p.G + g) * p.cap + entry) * V;
      for (int d = lane; d < V; d += 64) {
        const float x = ld(row + c0 + d) + (p.bias ? p.bias[c0 + d] : 0.f);
        st(row + c0 + d, x);
        if (keep) st(v + d, x);
      }
    }
  }
}

// The same for head sizes that are multiples of 4: four elements (two pairs) a lane, L lanes a head, so a
// wave works on 64 / L heads at once.
template <typename T, int L>
__global__ void __launch_bounds__(256) attn_prep4_kernel(WindowAttnParams p) {
  constexpr int HPB = 256 / L;   // heads at once
  const int64_t m = blockIdx.x;
  const int b = (int)(m / p.T), t = (int)(m % p.T);
  const int len = p.lens ? min(p.lens[b], p.T) : p.T;
  if (t >= len) return;
  const int64_t ps = pos_of(p.pos, p.pos_stride, b) + t;
  const int64_t pt = ps < p.max_pos ? ps : p.max_pos - 1;
  const int slot = slot_of(p.slots, b, p.nslots);
  const int entry = (int)(ps % p.cap);
  const bool keep = t >= len - p.cap;   // a prompt longer than the ring: only its last entries
  T* row = static_cast<T*>(p.buf) + m * p.ldb;
  const int nq = p.H * p.maps, nk = p.G * p.maps, D = p.D, V = p.V, half = p.rot / 2;
  const int d = (threadIdx.x % L) * 4;
  const bool ok = d < D;
  const float *cs = p.cos_t + pt * half, *sn = p.sin_t + pt * half;
  float c2[2] = {1.f, 1.f}, s2[2] = {0.f, 0.f};
#pragma unroll
  for (int i = 0; i < 2; ++i)
    if (d / 2 + i < half) c2[i] = cs[d / 2 + i], s2[i] = sn[d / 2 + i];
  const f32x4_t zero = {0.f, 0.f, 0.f, 0.f}, one = {1.f, 1.f, 1.f, 1.f};
  for (int h0 = 0; h0 < nq + nk; h0 += HPB) {   // (uniform: the reduction needs every lane)
    const int hd = h0 + threadIdx.x / L;
    const bool in = ok && hd < nq + nk;
    T* x = row + hd * D + d;
    f32x4_t v = in ? ld4(x) : zero;
    if (in && p.bias) v += ld4(p.bias + hd * D + d);
    const f32x4_t w = in && p.qn_w ? ld4((hd < nq ? p.qn_w : p.kn_w) + d) : one;
    const float ss = sum_lanes<L>(v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3]);
    if (!in) continue;
    if (p.qn_w) v *= w * (1.f / sqrtf(ss / (float)D + p.eps));
    const f32x4_t o = {v[0] * c2[0] - v[1] * s2[0], v[1] * c2[0] + v[0] * s2[0], v[2] * c2[1] - v[3] * s2[1],
                       v[3] * c2[1] + v[2] * s2[1]};
    st4(x, o);
    if (hd >= nq && keep) st4(static_cast<T*>(p.kc) + (((int64_t)slot * nk + (hd - nq)) * p.cap + entry) * D + d, o);
  }
  const int c0 = (nq + nk) * D;
  for (int i = threadIdx.x * 4; i < p.G * V; i += 1024) {
    f32x4_t v = ld4(row + c0 + i);
    if (p.bias) {
      v += ld4(p.bias + c0 + i);
      st4(row + c0 + i, v);
    }
    if (keep) st4(static_cast<T*>(p.vc) + (((int64_t)slot * p.G + i / V) * p.cap + entry) * V + i % V, v);
  }
}

__device__ __forceinline__ float cap_score(float s, float scale, float cap) {
  s *= scale;
  return cap > 0.f ? cap * tanhf(s / cap) : s;
}

// where a head's keys and values are: entry j of either the step's buffer or the ring
template <typename T>
struct KeySource {
  const T *k, *v;
  int64_t ks, vs, kmap;   // strides between keys, and between a head's maps
  int mod;
  __device__ KeySource(const WindowAttnParams& p, int b, int g) {
    if (p.from_buf) {
      k = static_cast<const T*>(p.kbuf) + (int64_t)b * p.T * p.ldk + (int64_t)g * p.maps * p.D;
      v = static_cast<const T*>(p.vbuf) + (int64_t)b * p.T * p.ldv + (int64_t)g * p.V;
      ks = p.ldk;
      vs = p.ldv;
      kmap = p.D;
      mod = 0x7fffffff;
    } else {
      const int slot = slot_of(p.slots, b, p.nslots);
      k = static_cast<const T*>(p.kc) + ((int64_t)slot * p.G + g) * p.maps * p.cap * p.D;
      v = static_cast<const T*>(p.vc) + ((int64_t)slot * p.G + g) * p.cap * p.V;
      ks = p.D;
      vs = p.V;
      kmap = (int64_t)p.cap * p.D;
      mod = p.cap;
    }
  }
  struct Pooled {};
  __device__ KeySource(const WindowAttnParams& p, int b, int g, Pooled) {   // (one map)
    const int64_t head = (int64_t)slot_of(p.slots, b, p.nslots) * p.G + g;
    k = static_cast<const T*>(p.pk) + head * p.pcap * p.D;
    v = static_cast<const T*>(p.pv) + head * p.pcap * p.V;
    ks = p.D;
    vs = p.V;
    kmap = 0;
    mod = 0x7fffffff;
  }
};

// Attention of one query (all maps of one head) over keys [j0, j1) by one wave: keys across lanes for
// the scores, value columns across lanes for the sums.  `q` [MAPS][D] and `pw` [MAPS][64] are the
// wave's LDS.  acc holds columns lane, lane + 64, ...; m / l the running maximum and weight sum.
template <typename T, int MAPS, int VC>
__device__ __forceinline__ void attend(const WindowAttnParams& p, const KeySource<T>& src, const float* q, float* pw,
                                       int64_t j0, int64_t j1, float (&acc)[MAPS][VC], float (&mx)[MAPS],
                                       float (&ls)[MAPS]) {
  const int lane = threadIdx.x & 63, D = p.D, V = p.V;
  for (int64_t base = j0; base < j1; base += 64) {
    const int n = (int)min((int64_t)64, j1 - base);
    const int64_t e = (base + min(lane, n - 1)) % src.mod;
#pragma unroll
    for (int c = 0; c < MAPS; ++c) {
      const T* kr = src.k + e * src.ks + c * src.kmap;
      float s = 0.f;
      for (int d = 0; d < D; ++d) s += ld(kr + d) * q[c * D + d];
      s = lane < n ? cap_score(s, p.scale, p.softcap) : -INFINITY;
      const float m2 = fmaxf(mx[c], wave_max(s));
      const float f = expf(mx[c] - m2), w = lane < n ? expf(s - m2) : 0.f;
      mx[c] = m2;
      ls[c] = ls[c] * f + wave_sum(w);
      pw[c * 64 + lane] = w;
#pragma unroll
      for (int i = 0; i < VC; ++i) acc[c][i] *= f;
    }
    __builtin_amdgcn_wave_barrier();
    for (int j = 0; j < n; ++j) {
      const T* vr = src.v + ((base + j) % src.mod) * src.vs;
#pragma unroll
      for (int i = 0; i < VC; ++i) {
        const int d = lane + 64 * i;
        if (d < V) {
          const float x = ld(vr + d);
#pragma unroll
          for (int c = 0; c < MAPS; ++c) acc[c][i] += pw[c * 64 + j] * x;
        }
      }
    }
    __builtin_amdgcn_wave_barrier();
  }
}

// the head's output from its maps' normalised outputs a[map][column]
template <typename T, int MAPS, int VC>
__device__ __forceinline__ void finish_head(const WindowAttnParams& p, int64_t m, int h, float (&a)[MAPS][VC]) {
  const int lane = threadIdx.x & 63, V = p.V;
  float r = p.out_scale;
  if constexpr (MAPS == 2) {
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < VC; ++i) {
      a[0][i] -= p.lam * a[1][i];
      if (lane + 64 * i < V) ss += a[0][i] * a[0][i];
    }
    r = p.out_scale / sqrtf(wave_sum(ss) / (float)V + p.out_eps);
  }
  T* y = static_cast<T*>(p.y) + m * p.ldy + (int64_t)h * V;
#pragma unroll
  for (int i = 0; i < VC; ++i)
    if (lane + 64 * i < V) st(y + lane + 64 * i, a[0][i] * r);
}

template <typename T, int MAPS, int VC>
__global__ void __launch_bounds__(256) attn_row_kernel(WindowAttnParams p) {
  extern __shared__ __attribute__((aligned(16))) float smem[];
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, D = p.D;
  float* q = smem + wid * (MAPS * D + MAPS * 64);
  float* pw = q + MAPS * D;
  const int64_t item = (int64_t)blockIdx.x * 4 + wid;
  if (item >= (int64_t)p.B * p.T * p.H) return;   // waves are independent: no block barrier below
  const int64_t m = item / p.H;
  const int h = (int)(item % p.H), b = (int)(m / p.T), t = (int)(m % p.T), g = h / (p.H / p.G);
  if (p.lens && t >= p.lens[b]) {
    T* y = static_cast<T*>(p.y) + m * p.ldy + (int64_t)h * p.V;
    for (int d = lane; d < p.V; d += 64) st(y + d, 0.f);
    return;
  }
  const T* qr = static_cast<const T*>(p.buf) + m * p.ldb + (int64_t)h * MAPS * D;
  for (int i = lane; i < MAPS * D; i += 64) q[i] = ld(qr + i);
  __builtin_amdgcn_wave_barrier();
  const int64_t ps = p.from_buf ? t : pos_of(p.pos, p.pos_stride, b) + t;
  const int64_t j0 = p.window > 0 && ps - p.window + 1 > 0 ? ps - p.window + 1 : 0;
  float acc[MAPS][VC] = {}, mx[MAPS], ls[MAPS];
#pragma unroll
  for (int c = 0; c < MAPS; ++c) mx[c] = -INFINITY, ls[c] = 0.f;
  if constexpr (MAPS == 1) {
    if (p.pool > 0)
      attend<T, MAPS, VC>(p, KeySource<T>(p, b, g, typename KeySource<T>::Pooled()), q, pw, 0, blocks_seen(p, ps), acc, mx, ls);
  }
  attend<T, MAPS, VC>(p, KeySource<T>(p, b, g), q, pw, j0, ps + 1, acc, mx, ls);
#pragma unroll
  for (int c = 0; c < MAPS; ++c)
#pragma unroll
    for (int i = 0; i < VC; ++i) acc[c][i] /= ls[c];
  finish_head<T, MAPS, VC>(p, m, h, acc);
}

template <typename T, int MAPS>
static int run_row(const WindowAttnParams& p, hipStream_t s) {
  const dim3 grid((unsigned)ceil_div64((int64_t)p.B * p.T * p.H, 4));
  const size_t lds = 4 * (size_t)MAPS * (p.D + 64) * 4;
  switch ((p.V + 63) / 64) {
    case 1: hipLaunchKernelGGL((attn_row_kernel<T, MAPS, 1>), grid, dim3(256), lds, s, p); break;
    case 2: hipLaunchKernelGGL((attn_row_kernel<T, MAPS, 2>), grid, dim3(256), lds, s, p); break;
    case 3: hipLaunchKernelGGL((attn_row_kernel<T, MAPS, 3>), grid, dim3(256), lds, s, p); break;
    case 4: hipLaunchKernelGGL((attn_row_kernel<T, MAPS, 4>), grid, dim3(256), lds, s, p); break;
    default: return -1;
  }
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

}  // namespace hybrid

template <typename T>
static int run_prep(const WindowAttnParams& p, hipStream_t s) {
  using namespace hybrid;
  const dim3 grid((unsigned)(p.B * p.T)), block(256);
  if (p.D % 4 || p.V % 4 || p.ldb % 4 || reinterpret_cast<uintptr_t>(p.buf) % 16)
    hipLaunchKernelGGL((attn_prep_kernel<T>), grid, block, 0, s, p);
  else if (p.D <= 16) hipLaunchKernelGGL((attn_prep4_kernel<T, 4>), grid, block, 0, s, p);
  else if (p.D <= 32) hipLaunchKernelGGL((attn_prep4_kernel<T, 8>), grid, block, 0, s, p);
  else if (p.D <= 64) hipLaunchKernelGGL((attn_prep4_kernel<T, 16>), grid, block, 0, s, p);
  else if (p.D <= 128) hipLaunchKernelGGL((attn_prep4_kernel<T, 32>), grid, block, 0, s, p);
  else hipLaunchKernelGGL((attn_prep4_kernel<T, 64>), grid, block, 0, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

int attn_prep_launch(bool f32, const WindowAttnParams& p, hipStream_t s) {
  return f32 ? run_prep<float>(p, s) : run_prep<uint16_t>(p, s);
}

int attn_prompt_d32_launch(const WindowAttnParams&, hipStream_t);
int attn_prompt_d48_launch(const WindowAttnParams&, hipStream_t);
int attn_prompt_d64_launch(const WindowAttnParams&, hipStream_t);
int attn_prompt_d96_launch(const WindowAttnParams&, hipStream_t);
int attn_prompt_d128_launch(const WindowAttnParams&, hipStream_t);

// bf16 prompts on the matrix cores: 16-byte pieces of every head, head sizes the kernels are built for
bool attn_prompt_supported(const WindowAttnParams& p) {
  return p.from_buf && p.T > 1 && p.D <= 128 && p.V <= 256 && p.D % 8 == 0 && p.V % 8 == 0 && p.ldb % 8 == 0 &&
         p.ldk % 8 == 0 && p.ldv % 8 == 0 && p.ldy % 4 == 0 && reinterpret_cast<uintptr_t>(p.buf) % 16 == 0 &&
         reinterpret_cast<uintptr_t>(p.kbuf) % 16 == 0 && reinterpret_cast<uintptr_t>(p.vbuf) % 16 == 0 &&
         reinterpret_cast<uintptr_t>(p.y) % 8 == 0;
}
int attn_prompt_launch(const WindowAttnParams& p, hipStream_t s) {
  if (p.D <= 32) return attn_prompt_d32_launch(p, s);
  if (p.D <= 48) return attn_prompt_d48_launch(p, s);
  if (p.D <= 64) return attn_prompt_d64_launch(p, s);
  if (p.D <= 96) return attn_prompt_d96_launch(p, s);
  return attn_prompt_d128_launch(p, s);
}

int attn_row_launch(bool f32, const WindowAttnParams& p, hipStream_t s) {
  if (p.maps == 2) return f32 ? hybrid::run_row<float, 2>(p, s) : hybrid::run_row<uint16_t, 2>(p, s);
  if (p.maps == 1) return f32 ? hybrid::run_row<float, 1>(p, s) : hybrid::run_row<uint16_t, 1>(p, s);
  return -1;
}

}  // namespace nxd
