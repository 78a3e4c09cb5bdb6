// One new token per sequence: q / k preparation, cache write and attention in one launch.
//
// A workgroup takes 256 of the visible keys of one (sequence, head), 64 a wave: scores with a key a lane,
// then value columns four a lane.  Every workgroup prepares the head's query itself; the one that owns
// the new key prepares key and value too (the group's first head also stores them in the cache), so
// nothing waits for another launch.  With more than 256 visible keys the partial sums go to `part` and
// the last workgroup of the head to arrive (a ticket in `tickets`, left at zero) merges them in order.
#include "window_attn.h"

namespace nxd {
namespace hybrid {

// bias, RMS norm, rotary turn of one head by one wave; out [D], rounded to the activation type
template <typename T>
__device__ __forceinline__ void prepare_head(const WindowAttnParams& p, const T* x, const float* bias, const float* nw,
                                             int64_t pt, float* out) {
  const int lane = threadIdx.x & 63, D = p.D, half = p.rot / 2;
  float u[2], w[2], ss = 0.f;
#pragma unroll
  for (int i = 0; i < 2; ++i) {   // pair lane + 64 i
    const int d = 2 * (lane + 64 * i);
    u[i] = d < D ? ld(x + d) + (bias ? bias[d] : 0.f) : 0.f;
    w[i] = d + 1 < D ? ld(x + d + 1) + (bias ? bias[d + 1] : 0.f) : 0.f;
    ss += u[i] * u[i] + w[i] * w[i];
  }
  const float r = nw ? 1.f / sqrtf(sum64(ss) / (float)D + p.eps) : 1.f;
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

__device__ __forceinline__ float dot_row(const float* k, const float* q, int D) {
  float s = 0.f;
  for (int d = 0; d < D; ++d) s += k[d] * q[d];
  return s;
}
__device__ __forceinline__ float dot_row8(const uint16_t* k, const float* q, int D) {   // D % 8 == 0, aligned
  float s = 0.f, s2 = 0.f;
#pragma unroll 4
  for (int d = 0; d < D; d += 8) {
    float f[8];
    unpack8(*reinterpret_cast<const u32x4_t*>(k + d), f);
    const f32x4_t a = ld4(q + d), b = ld4(q + d + 4);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      s += f[i] * a[i];
      s2 += f[4 + i] * b[i];
    }
  }
  return s + s2;
}
__device__ __forceinline__ float dot_row8(const float* k, const float* q, int D) { return dot_row(k, q, D); }

// VEC: head sizes are multiples of 8 (16-byte key pieces, 4-column value pieces)
template <typename T, int MAPS, bool VEC>
__global__ void __launch_bounds__(256) attn_decode_kernel(WindowAttnParams p) {
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
  const int n = (int)(ps - j0 + 1);                     // visible keys, the new one last
  const T* row = static_cast<const T*>(p.buf) + (int64_t)b * p.ldb;
  const T* kc = static_cast<const T*>(p.kc) + ((int64_t)slot * p.G + g) * MAPS * p.cap * D;
  const T* vc = static_cast<const T*>(p.vc) + ((int64_t)slot * p.G + g) * p.cap * V;
  const int first = sp * 256, last = min(n, first + 256) - 1;
  const bool owner = first < n && last == n - 1;        // this workgroup has the new key

  if (first < n) {
    const int64_t qk0 = (int64_t)p.H * MAPS * D;
    for (int job = w; job < (owner ? 2 * MAPS + 1 : MAPS); job += 4) {
      if (job < MAPS) {
        const int64_t c = ((int64_t)h * MAPS + job) * D;
        prepare_head<T>(p, row + c, p.bias ? p.bias + c : nullptr, p.qn_w, pt, q[job]);
      } else if (job < 2 * MAPS) {
        const int m = job - MAPS;
        const int64_t c = qk0 + ((int64_t)g * MAPS + m) * D;
        prepare_head<T>(p, row + c, p.bias ? p.bias + c : nullptr, p.kn_w, pt, kn[m]);
      } else {
        const int64_t c = qk0 + (int64_t)p.G * MAPS * D + (int64_t)g * V;
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
  }

  // ---- this wave's 64 keys
  const int k0 = first + 64 * w, cnt = min(64, n - k0);
  float mx[MAPS], ls[MAPS];
#pragma unroll
  for (int c = 0; c < MAPS; ++c) mx[c] = -INFINITY, ls[c] = 0.f;
  for (int i = lane; i < MAPS * V; i += 64) acc[w][i / V][i % V] = 0.f;
  if (cnt > 0) {
    const int key = k0 + min(lane, cnt - 1);
    const int e = (int)((j0 + key) % p.cap);
#pragma unroll
    for (int c = 0; c < MAPS; ++c) {
      float s;
      if (key == n - 1) s = dot_row(kn[c], q[c], D);
      else if (VEC) s = dot_row8(kc + ((int64_t)c * p.cap + e) * D, q[c], D);
      else {
        const T* kr = kc + ((int64_t)c * p.cap + e) * D;
        s = 0.f;
        for (int d = 0; d < D; ++d) s += ld(kr + d) * q[c][d];
      }
      s *= p.scale;
      if (p.softcap > 0.f) s = p.softcap * tanhf(s / p.softcap);
      if (lane >= cnt) s = -INFINITY;
      mx[c] = wave_max(s);
      const float x = lane < cnt ? expf(s - mx[c]) : 0.f;
      ls[c] = sum64(x);
      pw[w][c][lane] = x;
    }
    __builtin_amdgcn_wave_barrier();
    if (VEC) {
      const int lpr = V <= 32 ? 8 : (V <= 64 ? 16 : (V <= 128 ? 32 : 64)), kpp = 64 / lpr;   // lanes a row, keys a pass
      const int col = (lane % lpr) * 4, ks = lane / lpr;
      f32x4_t a[MAPS];
#pragma unroll
      for (int c = 0; c < MAPS; ++c) a[c] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      if (col < V) {
#pragma unroll 8
        for (int j = 0; j < cnt; j += kpp) {
          const int i = min(j + ks, cnt - 1), key2 = k0 + i;
          const bool in = j + ks < cnt;
          const f32x4_t x = key2 == n - 1 ? ld4(vn + col) : ld4(vc + (int64_t)((j0 + key2) % p.cap) * V + col);
#pragma unroll
          for (int c = 0; c < MAPS; ++c) a[c] += x * (in ? pw[w][c][i] : 0.f);
        }
      }
#pragma unroll
      for (int c = 0; c < MAPS; ++c) {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          for (int o = lpr; o < 64; o <<= 1) a[c][i] += __shfl_xor(a[c][i], o, 64);
        if (ks == 0 && col < V) st4(&acc[w][c][col], a[c]);
      }
    } else {
      for (int d = lane; d < V; d += 64) {
        float a[MAPS] = {};
        for (int j = 0; j < cnt; ++j) {
          const int key2 = k0 + j;
          const float x = key2 == n - 1 ? vn[d] : ld(vc + (int64_t)((j0 + key2) % p.cap) * V + d);
#pragma unroll
          for (int c = 0; c < MAPS; ++c) a[c] += pw[w][c][j] * x;
        }
#pragma unroll
        for (int c = 0; c < MAPS; ++c) acc[w][c][d] = a[c];
      }
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
    if (tid == 0) arrival = __hip_atomic_fetch_add(p.tickets + head, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    __syncthreads();
    if (arrival != p.splits - 1) return;
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup");
    if (tid == 0) __hip_atomic_store(p.tickets + head, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
#pragma unroll
    for (int c = 0; c < MAPS; ++c) {
      m[c] = -INFINITY;
      l[c] = a[c] = 0.f;
      for (int s = 0; s < p.splits; ++s) {
        const float* o = p.part + (head * p.splits + s) * stride + c * (V + 2);
        const float ms = __hip_atomic_load(o, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        if (ms == -INFINITY) continue;   // a split past the visible keys
        const float lsum = __hip_atomic_load(o + 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        const float as = tid < V ? __hip_atomic_load(o + 2 + tid, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) : 0.f;
        const float m2 = fmaxf(m[c], ms), f = m[c] == -INFINITY ? 0.f : expf(m[c] - m2), fs = expf(ms - m2);
        l[c] = l[c] * f + lsum * fs;
        a[c] = a[c] * f + as * fs;
        m[c] = m2;
      }
    }
  }
  float o = a[0] / l[0];
  if constexpr (MAPS == 2) {
    o -= p.lam * (a[1] / l[1]);
    o *= p.out_scale / sqrtf(block_sum(tid < V ? o * o : 0.f, red) / (float)V + p.out_eps);
  }
  if (tid < V) st(static_cast<T*>(p.y) + (int64_t)b * p.ldy + (int64_t)h * V + tid, o);
}

template <typename T, int MAPS>
static int run_decode(const WindowAttnParams& p, hipStream_t s) {
  const dim3 grid((unsigned)p.splits, (unsigned)p.H, (unsigned)p.B);
  if (p.D % 8 == 0 && p.V % 8 == 0) hipLaunchKernelGGL((attn_decode_kernel<T, MAPS, true>), grid, dim3(256), 0, s, p);
  else hipLaunchKernelGGL((attn_decode_kernel<T, MAPS, false>), grid, dim3(256), 0, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

}  // namespace hybrid

int attn_decode_launch(bool f32, const WindowAttnParams& p, hipStream_t s) {
  if (p.maps == 2) return f32 ? hybrid::run_decode<float, 2>(p, s) : hybrid::run_decode<uint16_t, 2>(p, s);
  return f32 ? hybrid::run_decode<float, 1>(p, s) : hybrid::run_decode<uint16_t, 1>(p, s);
}

}  // namespace nxd
