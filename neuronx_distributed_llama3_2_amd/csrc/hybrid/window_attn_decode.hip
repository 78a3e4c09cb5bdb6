// One new token per sequence: q / k preparation, cache write and attention in one launch.
//
// A workgroup takes some of the visible keys of one (sequence, head): scores with a key a lane, then value
// columns four a lane.  Every workgroup prepares the head's query itself; the one that owns the new key
// prepares key and value too (the group's first head also stores them in the cache), so nothing waits for
// another launch.  With several workgroups a head the partial sums go to `part` and the last one to arrive
// (a ticket in `tickets`, left at zero) merges them in order.
//
// POOL: the pooled blocks that the query sees are the first of its keys, the window's follow; the workgroup
// that has a new key which ends a block writes the block's means (no query sees them before a later step).
#include "window_attn.h"

namespace nxd {
namespace hybrid {

// bias, RMS norm, rotary turn of one head by one wave; out [D], rounded to the activation type
template <typename T>
__device__ __forceinline__ void prepare_head(const WindowAttnParams& p, const T* x, const float* bias, const float* nw,
                                             int64_t pt, float* out, float row_r = 0.f) {
  const int lane = threadIdx.x & 63, D = p.D, half = p.rot / 2;
  float u[2], w[2], ss = 0.f;
#pragma unroll
  for (int i = 0; i < 2; ++i) {   // pair lane + 64 i
    const int d = 2 * (lane + 64 * i);
    u[i] = d < D ? ld(x + d) + (bias ? bias[d] : 0.f) : 0.f;
    w[i] = d + 1 < D ? ld(x + d + 1) + (bias ? bias[d + 1] : 0.f) : 0.f;
    ss += u[i] * u[i] + w[i] * w[i];
  }
  const float r = row_r > 0.f ? row_r : (nw ? 1.f / sqrtf(sum64(ss) / (float)D + p.eps) : 1.f);
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
    T t;
    st(&t, a);
    out[d] = ld(&t);
    if (d + 1 < D) {
      st(&t, c);
      out[d + 1] = ld(&t);
    }
  }
}

// 1 / sqrt(mean of squares + eps) of n elements, by every wave for itself
template <typename T>
__device__ __forceinline__ float row_rms(const T* x, int n, float eps) {
  const int lane = threadIdx.x & 63;
  float ss = 0.f;
  if (n % 4 == 0 && reinterpret_cast<uintptr_t>(x) % (4 * sizeof(T)) == 0) {
#pragma unroll 4
    for (int i = lane * 4; i < n; i += 256) {
      const f32x4_t v = ld4(x + i);
      ss += v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
    }
  } else {
    for (int i = lane; i < n; i += 64) {
      const float v = ld(x + i);
      ss += v * v;
    }
  }
  return 1.f / sqrtf(sum64(ss) / (float)n + eps);
}

// The means of the block that the new token (position ps, its key and value in LDS) ends, by 256 threads:
// thread = element of the row and slice of the tokens.  red: at least 4 x 256 floats of LDS; every thread of
// the workgroup calls it.
template <typename T>
__device__ __forceinline__ void pool_block(const WindowAttnParams& p, int slot, int g, int64_t ps, const float* kn, const float* vn,
                                           float* red) {
  const int tid = threadIdx.x, D = p.D;
  const int width = D <= 64 ? 64 : (D <= 128 ? 128 : 256), slices = 256 / width, d = tid % width, sl = tid / width;
  const int64_t head = (int64_t)slot * p.G + g, blk = ps / p.pool;
  if (blk >= p.pcap) return;
#pragma unroll
  for (int which = 0; which < 2; ++which) {   // D == V
    const T* src = static_cast<const T*>(which ? p.vc : p.kc) + head * p.cap * D;
    const float* last = which ? vn : kn;
    float a = 0.f;
    if (d < D) {
#pragma unroll 8
      for (int64_t t = ps - p.pool + 1 + sl; t < ps; t += slices) a += ld(src + (t % p.cap) * D + d);
    }
    __syncthreads();
    red[sl * 256 + d] = a;
    __syncthreads();
    if (sl == 0 && d < D) {
      for (int i = 1; i < slices; ++i) a += red[i * 256 + d];
      st(static_cast<T*>(which ? p.pv : p.pk) + (head * p.pcap + blk) * D + d, (a + last[d]) / (float)p.pool);
    }
  }
  __syncthreads();
}

// A workgroup's sums over its keys (thread = value column): merged with the head's other workgroups if
// there are any, combined over the maps and stored.
template <typename T, int MAPS>
__device__ __forceinline__ void finish(const WindowAttnParams& p, int b, int h, int sp, float (&m)[MAPS], float (&l)[MAPS],
                                       float (&a)[MAPS], float* red, int* arrival) {
  const int tid = threadIdx.x, V = p.V;
  if (p.splits > 1) {
    const int64_t head = (int64_t)b * p.H + h, stride = MAPS * (V + 2);
    float* part = p.part + (head * p.splits + sp) * stride;
#pragma unroll
    for (int c = 0; c < MAPS; ++c) {
      if (tid < V) __hip_atomic_store(part + c * (V + 2) + 2 + tid, a[c], __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
      if (tid == 0) {
        __hip_atomic_store(part + c * (V + 2), m[c], __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        __hip_atomic_store(part + c * (V + 2) + 1, l[c], __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
      }
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");   // every wave's stores have left before the ticket
    __syncthreads();
    if (tid == 0) *arrival = __hip_atomic_fetch_add(p.tickets + head, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    __syncthreads();
    if (*arrival != p.splits - 1) return;
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup");
    if (tid == 0) __hip_atomic_store(p.tickets + head, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
#pragma unroll
    for (int c = 0; c < MAPS; ++c) m[c] = -INFINITY, l[c] = a[c] = 0.f;
    for (int s0 = 0; s0 < p.splits; s0 += 8) {   // eight splits' partial sums per round trip
      float ms[MAPS][8], lsum[MAPS][8], as[MAPS][8];
#pragma unroll
      for (int i = 0; i < 8; ++i)
#pragma unroll
        for (int c = 0; c < MAPS; ++c) {
          const float* o = p.part + (head * p.splits + min(s0 + i, p.splits - 1)) * stride + c * (V + 2);
          ms[c][i] = __hip_atomic_load(o, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
          lsum[c][i] = __hip_atomic_load(o + 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
          as[c][i] = __hip_atomic_load(o + 2 + min(tid, V - 1), __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        }
#pragma unroll
      for (int i = 0; i < 8; ++i)
#pragma unroll
        for (int c = 0; c < MAPS; ++c) {
          if (s0 + i >= p.splits || ms[c][i] == -INFINITY) continue;   // (no split, or one past the visible keys)
          const float m2 = fmaxf(m[c], ms[c][i]), f = m[c] == -INFINITY ? 0.f : expf(m[c] - m2), fs = expf(ms[c][i] - m2);
          l[c] = l[c] * f + lsum[c][i] * fs;
          a[c] = a[c] * f + as[c][i] * fs;
          m[c] = m2;
        }
    }
  }
  float o = a[0] / l[0] * (MAPS == 1 ? p.out_scale : 1.f);
  if constexpr (MAPS == 2) {
    o -= p.lam * (a[1] / l[1]);
    o *= p.out_scale / sqrtf(block_sum(tid < V ? o * o : 0.f, red) / (float)V + p.out_eps);
  }
  if (tid < V) st(static_cast<T*>(p.y) + (int64_t)b * p.ldy + (int64_t)h * V + tid, o);
}

// ---- any head sizes: 256 keys a workgroup, 64 a wave
template <typename T, int MAPS, bool POOL>
__global__ void __launch_bounds__(256) attn_decode_any_kernel(WindowAttnParams p) {
  __shared__ __attribute__((aligned(16))) float q[MAPS][256], kn[MAPS][256], vn[256];
  __shared__ __attribute__((aligned(16))) float pw[4][MAPS][64], acc[4][MAPS][256];
  __shared__ float mw[4][MAPS], lw[4][MAPS], red[16];
  __shared__ int arrival;
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int sp = blockIdx.x, h = blockIdx.y, b = blockIdx.z, rep = p.H / p.G, g = h / rep, D = p.D, V = p.V;
  const int slot = slot_of(p.slots, b, p.nslots);
  const int64_t ps = pos_of(p.pos, p.pos_stride, b);
  const int64_t pt = ps < p.max_pos ? ps : p.max_pos - 1;
  int64_t j0 = p.window > 0 && ps - p.window + 1 > 0 ? ps - p.window + 1 : 0;
  if (ps - j0 >= p.cap) j0 = ps - p.cap + 1;            // the ring holds no more (a position beyond the cache)
  const int nb = POOL ? blocks_seen(p, ps) : 0;         // pooled blocks come first
  const int n = nb + (int)(ps - j0 + 1);                // visible keys, the new one last
  const T* row = static_cast<const T*>(p.buf) + (int64_t)b * p.ldb;
  const T* kc = static_cast<const T*>(p.kc) + ((int64_t)slot * p.G + g) * MAPS * p.cap * D;
  const T* vc = static_cast<const T*>(p.vc) + ((int64_t)slot * p.G + g) * p.cap * V;
  const int e0 = (int)(j0 % p.cap);                     // ring entry of key nb; key nb + i is e0 + i, wrapped once
  auto entry = [&](int i) { return e0 + i - nb >= p.cap ? e0 + i - nb - p.cap : e0 + i - nb; };
  const T* pk = static_cast<const T*>(p.pk) + (POOL ? ((int64_t)slot * p.G + g) * p.pcap * D : 0);
  const T* pv = static_cast<const T*>(p.pv) + (POOL ? ((int64_t)slot * p.G + g) * p.pcap * V : 0);
  const bool ends = POOL && (ps + 1) % p.pool == 0;     // the new token ends a block
  const int first = sp * 256, last = min(n, first + 256) - 1;
  const bool owner = first < n && last == n - 1;        // this workgroup has the new key

  if (first < n) {
    const int64_t qk0 = (int64_t)p.H * MAPS * D;
    float rq = 0.f, rk = 0.f;
    if (POOL && p.norm_all) {
      rq = row_rms(row, p.H * D, p.eps);
      if (owner) rk = row_rms(row + qk0, p.G * D, p.eps);
    }
    for (int job = w; job < (owner ? 2 * MAPS + 1 : MAPS); job += 4) {
      if (job < MAPS) {
        const int64_t c = ((int64_t)h * MAPS + job) * D;
        prepare_head<T>(p, row + c, p.bias ? p.bias + c : nullptr, p.norm_all ? p.qn_w + (int64_t)h * D : p.qn_w, pt, q[job], rq);
      } else if (job < 2 * MAPS) {
        const int m = job - MAPS;
        const int64_t c = qk0 + ((int64_t)g * MAPS + m) * D;
        prepare_head<T>(p, row + c, p.bias ? p.bias + c : nullptr, p.norm_all ? p.kn_w + (int64_t)g * D : p.kn_w, pt, kn[m], rk);
      } else {
        const int64_t c = p.v_off + (int64_t)g * V;
        for (int d = lane; d < V; d += 64) {
          T t;
          st(&t, ld(row + c + d) + (p.bias ? p.bias[c + d] : 0.f));
          vn[d] = ld(&t);
        }
      }
    }
  }
  __syncthreads();
  if (owner && h % rep == 0) {   // (the values are exact in the activation type)
    const int e = (int)(ps % p.cap);
    T* ko = static_cast<T*>(p.kc) + ((int64_t)slot * p.G + g) * MAPS * p.cap * D;
    T* vo = static_cast<T*>(p.vc) + ((int64_t)slot * p.G + g) * p.cap * V;
    for (int i = tid; i < MAPS * D; i += 256) st(ko + ((int64_t)(i / D) * p.cap + e) * D + i % D, kn[i / D][i % D]);
    for (int i = tid; i < V; i += 256) st(vo + (int64_t)e * V + i, vn[i]);
    if (ends) pool_block<T>(p, slot, g, ps, kn[0], vn, &acc[0][0][0]);
  }

  // ---- this wave's 64 keys
  const int k0 = first + 64 * w, cnt = min(64, n - k0);
  float mx[MAPS], ls[MAPS];
#pragma unroll
  for (int c = 0; c < MAPS; ++c) mx[c] = -INFINITY, ls[c] = 0.f;
  for (int i = lane; i < MAPS * V; i += 64) acc[w][i / V][i % V] = 0.f;
  if (cnt > 0) {
    const int key = k0 + min(lane, cnt - 1);
    const int e = POOL && key < nb ? 0 : entry(key);
    // the new key's entry may hold an old key or the new one by now: its score comes from LDS
    const bool has_new = k0 + cnt == n;
#pragma unroll
    for (int c = 0; c < MAPS; ++c) {
      float s;
      const T* kr = POOL && key < nb ? pk + (int64_t)key * D : kc + ((int64_t)c * p.cap + e) * D;
      s = 0.f;
      for (int d = 0; d < D; ++d) s += ld(kr + d) * q[c][d];
      if (has_new) {
        float t = 0.f;
        for (int d = lane; d < D; d += 64) t += kn[c][d] * q[c][d];
        t = sum64(t);
        if (key == n - 1) s = t;
      }
      s *= p.scale;
      if (p.softcap > 0.f) s = p.softcap * tanhf(s / p.softcap);
      if (lane >= cnt) s = -INFINITY;
      mx[c] = max64(s);
      const float x = lane < cnt ? expf(s - mx[c]) : 0.f;
      ls[c] = sum64(x);
      pw[w][c][lane] = x;
    }
    __builtin_amdgcn_wave_barrier();
    for (int d = lane; d < V; d += 64) {
      float a[MAPS] = {};
      for (int j = 0; j < cnt; ++j) {
        const int key2 = k0 + j;
        const float x = key2 == n - 1 ? vn[d] : (POOL && key2 < nb ? ld(pv + (int64_t)key2 * V + d) : ld(vc + (int64_t)entry(key2) * V + d));
#pragma unroll
        for (int c = 0; c < MAPS; ++c) a[c] += pw[w][c][j] * x;
      }
#pragma unroll
      for (int c = 0; c < MAPS; ++c) acc[w][c][d] = a[c];
    }
  }
  if (lane == 0) {
#pragma unroll
    for (int c = 0; c < MAPS; ++c) mw[w][c] = mx[c], lw[w][c] = ls[c];
  }
  __syncthreads();

  // ---- the workgroup's waves together: thread = value column
  float m[MAPS], l[MAPS], a[MAPS];
#pragma unroll
  for (int c = 0; c < MAPS; ++c) {
    m[c] = fmaxf(fmaxf(mw[0][c], mw[1][c]), fmaxf(mw[2][c], mw[3][c]));
    l[c] = a[c] = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float f = mw[i][c] == -INFINITY ? 0.f : expf(mw[i][c] - m[c]);
      l[c] += lw[i][c] * f;
      if (tid < V) a[c] += acc[i][c][tid] * f;
    }
  }
  finish<T, MAPS>(p, b, h, sp, m, l, a, red, &arrival);
}

// ---- head sizes that are multiples of 8, D <= 128: 64 keys a tile.  Keys and values of a tile are on
// their way before they are needed (the first tile's before the query is even prepared).  Neighbouring
// lanes read neighbouring pieces of a row: a key's score is a sum over LR lanes, a value row is spread
// over 8 to 64.  The keys of a map are shared by 4 / MAPS waves; every wave then has all 64 weights and
// sums 16 keys.
template <typename T>
struct Raw;
template <>
struct Raw<uint16_t> {
  typedef u32x2_t four;
  struct eight {
    u32x4_t v;
  };
};
template <>
struct Raw<float> {
  typedef f32x4_t four;
  struct eight {
    f32x4_t a, b;
  };
};
__device__ __forceinline__ f32x4_t widen(const u32x2_t& v) {
  return f32x4_t{__uint_as_float(v[0] << 16), __uint_as_float(v[0] & 0xffff0000u), __uint_as_float(v[1] << 16),
                 __uint_as_float(v[1] & 0xffff0000u)};
}
__device__ __forceinline__ f32x4_t widen(const f32x4_t& v) { return v; }
__device__ __forceinline__ float dot8(const Raw<uint16_t>::eight& k, const float (&q)[8]) {
  float f[8], s = 0.f;
  unpack8(k.v, f);
#pragma unroll
  for (int i = 0; i < 8; ++i) s += f[i] * q[i];
  return s;
}
__device__ __forceinline__ float dot8(const Raw<float>::eight& k, const float (&q)[8]) {
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) s += k.a[i] * q[i] + k.b[i] * q[4 + i];
  return s;
}

// R query heads of one key / value head share the keys and values a workgroup reads.  LR lanes of 8
// elements cover D.
template <typename T, int MAPS, int LR, int R, bool POOL>
__global__ void __launch_bounds__(256) attn_decode_kernel(WindowAttnParams p) {
  constexpr int PARTS = 4 / MAPS, RPL = 64 / LR, NK = (64 / PARTS) / RPL;   // waves a map, keys a load, loads a wave
  constexpr int NJ = R * MAPS, SM = (NJ + 3) / 4;                           // rows of weights, of them a wave
  static_assert(NK >= 1 && R <= 4, "whole loads, a wave a head at the end");
  typedef typename Raw<T>::four raw_t;
  __shared__ __attribute__((aligned(16))) float q[NJ][128], kn[MAPS][128], vn[256];
  __shared__ __attribute__((aligned(16))) float sc[2][NJ][64], pw[NJ][64], acc[4][NJ][256];
  __shared__ float fs[NJ], msum[NJ], lsum[NJ];
  __shared__ int arrival;
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int sp = blockIdx.x, h0 = blockIdx.y * R, b = blockIdx.z, rep = p.H / p.G, g = h0 / rep, D = p.D, V = p.V;
  const int slot = slot_of(p.slots, b, p.nslots);
  const int64_t ps = pos_of(p.pos, p.pos_stride, b);
  const int64_t pt = ps < p.max_pos ? ps : p.max_pos - 1;
  int64_t j0 = p.window > 0 && ps - p.window + 1 > 0 ? ps - p.window + 1 : 0;
  if (ps - j0 >= p.cap) j0 = ps - p.cap + 1;            // the ring holds no more (a position beyond the cache)
  const int nb = POOL ? blocks_seen(p, ps) : 0;         // pooled blocks come first
  const int n = nb + (int)(ps - j0 + 1);                // visible keys, the new one last
  const int e0 = (int)((uint32_t)j0 % (uint32_t)p.cap); // (positions are below 2^31)
  auto entry = [&](int i) { return e0 + i - nb >= p.cap ? e0 + i - nb - p.cap : e0 + i - nb; };
  const T* pk = static_cast<const T*>(p.pk) + (POOL ? ((int64_t)slot * p.G + g) * p.pcap * D : 0);
  const T* pv = static_cast<const T*>(p.pv) + (POOL ? ((int64_t)slot * p.G + g) * p.pcap * V : 0);
  const bool ends = POOL && (ps + 1) % p.pool == 0;     // the new token ends a block
  const T* row = static_cast<const T*>(p.buf) + (int64_t)b * p.ldb;
  T* kc = static_cast<T*>(p.kc) + ((int64_t)slot * p.G + g) * MAPS * p.cap * D;
  T* vc = static_cast<T*>(p.vc) + ((int64_t)slot * p.G + g) * p.cap * V;
  const int first = sp * p.tiles * 64, end = min(n, first + p.tiles * 64);
  const bool owner = first < n && end == n;             // this workgroup has the new key

  // this wave's map and keys of the scores, and its columns of the sums
  const int c = w % MAPS, part = w / MAPS, dl = (lane % LR) * 8, kl = lane / LR;
  const bool dok = dl < D;
  const int lpr = V <= 32 ? 8 : (V <= 64 ? 16 : (V <= 128 ? 32 : 64)), kpp = 64 / lpr;   // lanes a value row, rows a load
  const int col = min((lane % lpr) * 4, V - 4), ks = lane / lpr;
  typename Raw<T>::eight kr[NK];
  raw_t vr[16];
  auto fetch_k = [&](int k0) {   // (keys past the end re-read the last)
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int k = min(k0 + part * (64 / PARTS) + i * RPL + kl, n - 1);
      const T* src = POOL && k < nb ? pk + (int64_t)k * D : kc + ((int64_t)c * p.cap + entry(k)) * D;
      kr[i] = *reinterpret_cast<const typename Raw<T>::eight*>(src + (dok ? dl : 0));
    }
  };
  auto fetch_v = [&](int k0) {
#pragma unroll
    for (int i = 0; i < 16; ++i)
      if (i * kpp < 16) {
        const int k = min(k0 + 16 * w + i * kpp + ks, n - 1);
        vr[i] = *reinterpret_cast<const raw_t*>((POOL && k < nb ? pv + (int64_t)k * V : vc + (int64_t)entry(k) * V) + col);
      }
  };
  if (first < n) {
    fetch_k(first);
    fetch_v(first);
    const int64_t qk0 = (int64_t)p.H * MAPS * D;
    float rq = 0.f, rk = 0.f;
    if (POOL && p.norm_all) {
      rq = row_rms(row, p.H * D, p.eps);
      if (owner) rk = row_rms(row + qk0, p.G * D, p.eps);
    }
    for (int job = w; job < (owner ? NJ + MAPS + 1 : NJ); job += 4) {
      if (job < NJ) {
        const int64_t o = ((int64_t)h0 * MAPS + job) * D;
        prepare_head<T>(p, row + o, p.bias ? p.bias + o : nullptr, POOL && p.norm_all ? p.qn_w + o : p.qn_w, pt, q[job], rq);
      } else if (job < NJ + MAPS) {
        const int64_t o = qk0 + ((int64_t)g * MAPS + job - NJ) * D;
        prepare_head<T>(p, row + o, p.bias ? p.bias + o : nullptr, POOL && p.norm_all ? p.kn_w + (int64_t)g * D : p.kn_w, pt,
                        kn[job - NJ], rk);
      } else {
        const int64_t o = p.v_off + (int64_t)g * V;
        for (int d = lane; d < V; d += 64) {
          T t;
          st(&t, ld(row + o + d) + (p.bias ? p.bias[o + d] : 0.f));
          vn[d] = ld(&t);
        }
      }
    }
  }
  __syncthreads();
  if (owner && h0 % rep == 0) {   // (the values are exact in the activation type)
    const int e = entry(n - 1);
    for (int i = tid; i < MAPS * D; i += 256) st(kc + ((int64_t)(i / D) * p.cap + e) * D + i % D, kn[i / D][i % D]);
    for (int i = tid; i < V; i += 256) st(vc + (int64_t)e * V + i, vn[i]);
    if (ends) pool_block<T>(p, slot, g, ps, kn[0], vn, &acc[0][0][0]);
  }

  float q8[R][8], snew[R];   // this lane's piece of the queries; the new key's scores
#pragma unroll
  for (int r = 0; r < R; ++r) {
    snew[r] = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) q8[r][i] = dok ? q[r * MAPS + c][dl + i] : 0.f;
    if (owner) {
#pragma unroll
      for (int i = 0; i < 8; ++i) snew[r] += dok ? kn[c][dl + i] * q8[r][i] : 0.f;
      snew[r] = sum_lanes<LR>(snew[r]);
    }
  }
  float mx[SM], ls[SM];   // of weight rows w, w + 4
  f32x4_t a4[NJ];
#pragma unroll
  for (int i = 0; i < SM; ++i) mx[i] = -INFINITY, ls[i] = 0.f;
#pragma unroll
  for (int j = 0; j < NJ; ++j) a4[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  int flip = 0;
  for (int k0 = first; k0 < end; k0 += 64, flip ^= 1) {
    const int cnt = min(64, end - k0);
    const bool has_new = k0 + cnt == n;   // its entry may hold an old key or the new one by now: taken from LDS
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int k = part * (64 / PARTS) + i * RPL + kl;
#pragma unroll
      for (int r = 0; r < R; ++r) {
        float s = sum_lanes<LR>(dot8(kr[i], q8[r]));
        if (has_new && k == cnt - 1) s = snew[r];
        if (lane % LR == 0) sc[flip][r * MAPS + c][k] = s;
      }
    }
    if (k0 + 64 < end) fetch_k(k0 + 64);
    lds_barrier();   // (two score buffers: the next tile's scores do not wait for this one's readers)
#pragma unroll
    for (int i = 0; i < SM; ++i) {
      const int j = w + 4 * i;
      if (j < NJ) {
        float s = sc[flip][j][lane] * p.scale;
        if (p.softcap > 0.f) s = p.softcap * tanhf(s / p.softcap);
        if (lane >= cnt) s = -INFINITY;
        const float m2 = fmaxf(mx[i], max64(s));
        const float f = mx[i] == -INFINITY ? 0.f : expf(mx[i] - m2), x = lane < cnt ? expf(s - m2) : 0.f;
        mx[i] = m2;
        ls[i] = ls[i] * f + sum64(x);
        pw[j][lane] = x;
        if (lane == 0) fs[j] = f;
      }
    }
    lds_barrier();
#pragma unroll
    for (int j = 0; j < NJ; ++j) a4[j] *= fs[j];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      if (i * kpp < 16) {
        const int k = 16 * w + i * kpp + ks;
        f32x4_t x = widen(vr[i]);
        if (has_new && k >= cnt - 1) x = ld4(vn + col);   // (past the end: any finite value, its weight is zero)
#pragma unroll
        for (int j = 0; j < NJ; ++j) a4[j] += x * pw[j][k];
      }
    }
    if (k0 + 64 < end) fetch_v(k0 + 64);
  }
#pragma unroll
  for (int j = 0; j < NJ; ++j) {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      for (int o = lpr; o < 64; o <<= 1) a4[j][i] += __shfl_xor(a4[j][i], o, 64);
    if (ks == 0 && (lane % lpr) * 4 < V) st4(&acc[w][j][col], a4[j]);
  }
  if (lane == 0) {
#pragma unroll
    for (int i = 0; i < SM; ++i)
      if (w + 4 * i < NJ) msum[w + 4 * i] = mx[i], lsum[w + 4 * i] = ls[i];
  }
  __syncthreads();

  // ---- wave r finishes head h0 + r: columns lane, lane + 64, ...
  float l[MAPS], a[MAPS][4];
  const int hd = b * (p.H / R) + blockIdx.y, stride = NJ * (V + 2);
  if (p.splits > 1) {
    float* part_ = p.part + ((int64_t)hd * p.splits + sp) * stride;
    for (int i = tid; i < NJ * V; i += 256) {
      const int j = i / V, v = i % V;
      __hip_atomic_store(part_ + j * (V + 2) + 2 + v, acc[0][j][v] + acc[1][j][v] + acc[2][j][v] + acc[3][j][v], __ATOMIC_RELAXED,
                         __HIP_MEMORY_SCOPE_AGENT);
    }
    if (tid < NJ) {
      __hip_atomic_store(part_ + tid * (V + 2), msum[tid], __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
      __hip_atomic_store(part_ + tid * (V + 2) + 1, lsum[tid], __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");   // every wave's stores have left before the ticket
    __syncthreads();
    if (tid == 0) arrival = __hip_atomic_fetch_add(p.tickets + hd, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    __syncthreads();
    if (arrival != p.splits - 1) return;
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup");
    if (tid == 0) __hip_atomic_store(p.tickets + hd, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    if (w >= R) return;
    float m[MAPS];
#pragma unroll
    for (int k = 0; k < MAPS; ++k) {
      m[k] = -INFINITY;
      l[k] = 0.f;
#pragma unroll
      for (int i = 0; i < 4; ++i) a[k][i] = 0.f;
    }
    for (int s0 = 0; s0 < p.splits; s0 += 8) {   // eight splits' partial sums per round trip
      float ms[MAPS][8], lp[MAPS][8], as[MAPS][8][4];
#pragma unroll
      for (int s = 0; s < 8; ++s)
#pragma unroll
        for (int k = 0; k < MAPS; ++k) {
          const float* o = p.part + ((int64_t)hd * p.splits + min(s0 + s, p.splits - 1)) * stride + (w * MAPS + k) * (V + 2);
          ms[k][s] = __hip_atomic_load(o, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
          lp[k][s] = __hip_atomic_load(o + 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
#pragma unroll
          for (int i = 0; i < 4; ++i)
            as[k][s][i] = i == 0 || 64 * i < V ? __hip_atomic_load(o + 2 + min(lane + 64 * i, V - 1), __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) : 0.f;
        }
#pragma unroll
      for (int s = 0; s < 8; ++s)
#pragma unroll
        for (int k = 0; k < MAPS; ++k) {
          if (s0 + s >= p.splits || ms[k][s] == -INFINITY) continue;   // (no split, or one past the visible keys)
          const float m2 = fmaxf(m[k], ms[k][s]), f = m[k] == -INFINITY ? 0.f : expf(m[k] - m2), f2 = expf(ms[k][s] - m2);
          l[k] = l[k] * f + lp[k][s] * f2;
#pragma unroll
          for (int i = 0; i < 4; ++i) a[k][i] = a[k][i] * f + as[k][s][i] * f2;
          m[k] = m2;
        }
    }
  } else {
    if (w >= R) return;
#pragma unroll
    for (int k = 0; k < MAPS; ++k) {
      const int j = w * MAPS + k;
      l[k] = lsum[j];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int v = min(lane + 64 * i, V - 1);
        a[k][i] = acc[0][j][v] + acc[1][j][v] + acc[2][j][v] + acc[3][j][v];
      }
    }
  }
  float o[4], ss = 0.f, sc_out = p.out_scale;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    o[i] = a[0][i] / l[0];
    if constexpr (MAPS == 2) o[i] -= p.lam * (a[MAPS - 1][i] / l[MAPS - 1]);
    if (lane + 64 * i < V) ss += o[i] * o[i];
  }
  if constexpr (MAPS == 2) sc_out = p.out_scale / sqrtf(sum64(ss) / (float)V + p.out_eps);
  T* y = static_cast<T*>(p.y) + (int64_t)b * p.ldy + (int64_t)(h0 + w) * V;
#pragma unroll
  for (int i = 0; i < 4; ++i)
    if (lane + 64 * i < V) st(y + lane + 64 * i, o[i] * sc_out);
}

template <typename T, int MAPS, int R, bool POOL>
static void launch_decode(const WindowAttnParams& p, hipStream_t s) {
  const dim3 grid((unsigned)p.splits, (unsigned)(p.H / R), (unsigned)p.B);
  if (p.D <= 32) hipLaunchKernelGGL((attn_decode_kernel<T, MAPS, 4, R, POOL>), grid, dim3(256), 0, s, p);
  else if (p.D <= 64) hipLaunchKernelGGL((attn_decode_kernel<T, MAPS, 8, R, POOL>), grid, dim3(256), 0, s, p);
  else hipLaunchKernelGGL((attn_decode_kernel<T, MAPS, 16, R, POOL>), grid, dim3(256), 0, s, p);
}

template <typename T, int MAPS, bool POOL>
static int run_decode(const WindowAttnParams& p, hipStream_t s) {
  if (p.tiles == 0)
    hipLaunchKernelGGL((attn_decode_any_kernel<T, MAPS, POOL>), dim3((unsigned)p.splits, (unsigned)p.H, (unsigned)p.B), dim3(256), 0, s, p);
  else if (p.share == 4) launch_decode<T, MAPS, 4, POOL>(p, s);
  else if (p.share == 2) launch_decode<T, MAPS, 2, POOL>(p, s);
  else launch_decode<T, MAPS, 1, POOL>(p, s);
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

}  // namespace hybrid

// heads a workgroup takes, workgroups per such group and 64-key tiles each (0: the any-size kernel) for at
// most `seen` visible keys
void attn_decode_plan(WindowAttnParams& p, int64_t seen) {
  const int rep = p.H / p.G;
  if (p.D % 8 == 0 && p.V % 8 == 0 && p.D <= 128) {
    // heads share a workgroup's keys once there are enough workgroups without that (16 heads, 1,024 visible
    // keys, us with 1 / 4 heads a workgroup: 1 sequence 13 / 20, 16 sequences 31 / 25, 32 sequences 49 / 33)
    const int64_t all = (int64_t)p.B * p.H;
    p.share = all >= 256 && rep % 4 == 0 ? 4 : (all >= 128 && rep % 2 == 0 ? 2 : 1);
    // about 512 workgroups, but not more than 8 a group before each has 4 tiles: the merge has its price
    const int64_t tiles = (seen + 63) / 64, groups = (int64_t)p.B * p.H / p.share;
    const int64_t most = tiles / 4 > 8 ? tiles / 4 : (tiles < 8 ? tiles : 8);
    int64_t splits = 512 / groups;
    splits = splits < 1 ? 1 : (splits > most ? most : splits);
    p.tiles = (int)((tiles + splits - 1) / splits);
    p.splits = (int)((tiles + p.tiles - 1) / p.tiles);
  } else {
    p.share = 1;
    p.tiles = 0;
    p.splits = (int)((seen + 255) / 256);
  }
}

int attn_decode_launch(bool f32, const WindowAttnParams& p, hipStream_t s) {
  using namespace hybrid;
  if (p.pool > 0) return p.maps != 1 ? -1 : (f32 ? run_decode<float, 1, true>(p, s) : run_decode<uint16_t, 1, true>(p, s));
  if (p.maps == 2) return f32 ? run_decode<float, 2, false>(p, s) : run_decode<uint16_t, 2, false>(p, s);
  return f32 ? run_decode<float, 1, false>(p, s) : run_decode<uint16_t, 1, false>(p, s);
}

}  // namespace nxd
