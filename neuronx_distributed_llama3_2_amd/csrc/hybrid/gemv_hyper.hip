// Decode projections (1 to 4 rows) of hyper-connected decoders, with the element-wise work around them:
//
//   NORM prologue : x = rms_normalise(u) (1 + norm_w) from the fp32 sublayer input u [M, K]
//   epilogues     : store (bf16) | squared ReLU (bf16) | fp32 with a factor and an optional cap
//                   | HYPER: y + bias goes straight into the residual streams, x_t = sum_s mix[s][t] x_s +
//                   write[t] y, and u = sum_t read[t] x_t of the next sublayer comes out -- a column of
//                   the streams belongs to the one wave that owns the weight row, so it is updated in place
//
// So a sublayer is three launches: norm + projection, mixer (or nothing), projection + streams.
//
// Decode streams every weight byte once: a wave per weight row (or a K slice of it), bf16 dot products, a
// round of weight loads in flight before the prologue runs.  From 5 rows on the library's matrix products
// and hyper_step are faster (Golitar bench model of width 2048, ms per step, fused / not: 2 rows 0.98 /
// 1.48, 8 rows on a matrix-core form of this kernel 1.72 / 1.40).
#include "gemv_hyper.h"

namespace nxd {

namespace hybrid {

enum GemvEpi { STORE = 0, RELU2 = 1, F32CAP = 2, HYPER = 3 };

// the streams' old values of row m, column n: fetched ahead of the product
__device__ __forceinline__ void load_streams(const GemvHyperParams& p, int m, int n, float (&old)[8]) {
  const float* x = p.streams + (int64_t)m * p.S * p.N + n;
#pragma unroll
  for (int s = 0; s < 8; ++s) old[s] = s < p.S ? x[(int64_t)s * p.N] : 0.f;
}

// one output value of row m, column n
template <int EPI>
__device__ __forceinline__ void emit(const GemvHyperParams& p, int m, int n, float v, const float (&old)[8]) {
  if (EPI == STORE) {
    static_cast<uint16_t*>(p.y)[(int64_t)m * p.ldy + n] = f2bf(v);
  } else if (EPI == RELU2) {
    const float r = fmaxf(v, 0.f);
    static_cast<uint16_t*>(p.y)[(int64_t)m * p.ldy + n] = f2bf(r * r);
  } else if (EPI == F32CAP) {
    v *= p.alpha;
    static_cast<float*>(p.y)[(int64_t)m * p.ldy + n] = p.cap > 0.f ? p.cap * tanhf(v / p.cap) : v;
  } else {
    v = bf2f(f2bf(v)) + (p.bias ? p.bias[n] : 0.f);   // the projection's output is a bf16 activation
    float* x = p.streams + (int64_t)m * p.S * p.N + n;
    float u = 0.f;
#pragma unroll
    for (int t = 0; t < 8; ++t) {
      if (t >= p.S) break;
      float a = p.write[t] * v;
#pragma unroll
      for (int s = 0; s < 8; ++s)
        if (s < p.S) a += p.mix[s * p.S + t] * old[s];
      x[(int64_t)t * p.N] = a;
      u += p.read[t] * a;
    }
    p.un[(int64_t)m * p.N + n] = u;
  }
}

// normalised rows -> LDS (bf16) by a workgroup of NT threads; `first` holds columns tid 8 .. of row m,
// loaded ahead of the weights
template <int MM, int NT>
__device__ __forceinline__ void norm_rows(const GemvHyperParams& p, uint16_t* xs, float (*red)[MM], const f32x4_t (*first)[2]) {
  constexpr int NW = NT / 64;
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
#pragma unroll
  for (int m = 0; m < MM; ++m) {
    float ss = 0.f;
    if (m < p.M) {
      for (int k = tid * 8; k < p.K; k += NT * 8) {
        f32x4_t a, c;
        if (k == tid * 8) a = first[m][0], c = first[m][1];
        else a = ld4(p.u + (int64_t)m * p.K + k), c = ld4(p.u + (int64_t)m * p.K + k + 4);
#pragma unroll
        for (int i = 0; i < 4; ++i) ss += a[i] * a[i] + c[i] * c[i];
      }
    }
    ss = sum64(ss);
    if (lane == 0) red[wid][m] = ss;
  }
  __syncthreads();
  float rstd[MM];
#pragma unroll
  for (int m = 0; m < MM; ++m) {
    float t = 0.f;
#pragma unroll
    for (int i = 0; i < NW; ++i) t += red[i][m];
    rstd[m] = 1.f / sqrtf(t / (float)p.K + p.eps);
  }
  for (int k = tid * 8; k < p.K; k += NT * 8) {
    const f32x4_t g0 = ld4(p.norm_w + k), g1 = ld4(p.norm_w + k + 4);
#pragma unroll
    for (int m = 0; m < MM; ++m) {
      if (m < p.M) {
        f32x4_t a, c;
        if (k == tid * 8) a = first[m][0], c = first[m][1];
        else a = ld4(p.u + (int64_t)m * p.K + k), c = ld4(p.u + (int64_t)m * p.K + k + 4);
        float f[8];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          f[i] = a[i] * rstd[m] * (1.f + g0[i]);
          f[4 + i] = c[i] * rstd[m] * (1.f + g1[i]);
        }
        *reinterpret_cast<u32x4_t*>(xs + m * p.K + k) = pack8(f);
      }
    }
  }
  __syncthreads();
}

// ---- 1 or 2 rows.  4 waves = (4 / KS) weight rows x KS slices of K.
// U 512-element steps of a load round.
template <int MM, bool NORM, int EPI, int KS, int U>
__global__ void __launch_bounds__(256) gemv_hyper_kernel(GemvHyperParams p) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  uint16_t* xs = reinterpret_cast<uint16_t*>(smem);
  __shared__ float red[4][MM];
  __shared__ float part[4][MM];
  const int tid = threadIdx.x, lane = tid & 63, wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int n = blockIdx.x * (4 / KS) + wid / KS, ks = wid % KS;
  const uint16_t* wrow = p.w + (int64_t)min(n, p.N - 1) * p.ldw;
  const int kc = ((p.K + KS - 1) / KS + 7) & ~7;
  const int kbeg = min(ks * kc, p.K - 8), kend = max(kbeg + 8, min(p.K, ks * kc + kc));
  const bool some = ks * kc < p.K;
  f32x4_t first[MM][2];
  if constexpr (NORM) {   // ahead of the weights: loads retire in order
#pragma unroll
    for (int m = 0; m < MM; ++m) {
      const float* u = p.u + (int64_t)min(m, p.M - 1) * p.K + min(tid * 8, p.K - 8);
      first[m][0] = ld4(u);
      first[m][1] = ld4(u + 4);
    }
  }
  float old[8];
  if (EPI == HYPER && ks == 0 && lane < min(MM, p.M)) load_streams(p, lane, min(n, p.N - 1), old);
  u32x4_t wv[U], xv[NORM ? 1 : MM][U];
  auto load_x = [&](int base) {
    if constexpr (!NORM) {
#pragma unroll
      for (int m = 0; m < MM; ++m)
#pragma unroll
        for (int i = 0; i < U; ++i)
          xv[m][i] = *reinterpret_cast<const u32x4_t*>(p.x + (int64_t)min(m, p.M - 1) * p.ldx + min(base + i * 512 + lane * 8, kend - 8));
    }
  };
  auto load_round = [&](int base) {   // lanes past the end read the slice's last piece and skip it below
#pragma unroll
    for (int i = 0; i < U; ++i)
      wv[i] = __builtin_nontemporal_load(reinterpret_cast<const u32x4_t*>(wrow + min(base + i * 512 + lane * 8, kend - 8)));
  };
  load_x(kbeg);
  load_round(kbeg);
  if constexpr (NORM) norm_rows<MM, 256>(p, xs, red, first);
  float acc[MM];
#pragma unroll
  for (int m = 0; m < MM; ++m) acc[m] = 0.f;
  for (int base = kbeg; some && base < kend; base += 512 * U) {
    if (base != kbeg) {
      load_x(base);
      load_round(base);
    }
#pragma unroll
    for (int i = 0; i < U; ++i) {
      const int k = base + i * 512 + lane * 8;
      if (k < kend) {
#pragma unroll
        for (int m = 0; m < MM; ++m)
          if (m < p.M)
            acc[m] = dot8_bf16(NORM ? *reinterpret_cast<const u32x4_t*>(xs + m * p.K + k) : xv[NORM ? 0 : m][i], wv[i], acc[m]);
      }
    }
  }
#pragma unroll
  for (int m = 0; m < MM; ++m) acc[m] = sum64(acc[m]);
  if (KS > 1) {
    if (lane == 0) {
#pragma unroll
      for (int m = 0; m < MM; ++m) part[wid][m] = acc[m];
    }
    __syncthreads();
    if (ks != 0) return;
#pragma unroll
    for (int m = 0; m < MM; ++m)
#pragma unroll
      for (int i = 1; i < KS; ++i) acc[m] += part[wid + i][m];
  }
  if (n >= p.N || lane >= p.M || lane >= MM) return;
  float v = acc[0];
#pragma unroll
  for (int m = 1; m < MM; ++m) v = lane == m ? acc[m] : v;
  emit<EPI>(p, lane, n, v, old);   // lane m: row m
}

template <bool NORM, int EPI>
static int run_gemv(const GemvHyperParams& p, hipStream_t s) {
  const size_t lds = (size_t)p.M * p.K * 2;
  // K slices while the grid stays below 8,192 waves and a slice keeps 1,024 elements
  int ks = 1;
  while (ks < 4 && (int64_t)p.N * ks * 2 <= 8192 && p.K / (ks * 2) >= 1024) ks *= 2;
  const dim3 grid((unsigned)((p.N * ks + 3) / 4)), block(256);
#define NXD_GV(MMV, KSV, UV) hipLaunchKernelGGL((gemv_hyper_kernel<MMV, NORM, EPI, KSV, UV>), grid, block, NORM ? lds : 0, s, p)
#define NXD_GV_KS(MMV)                                       \
  if (ks == 1) NXD_GV(MMV, 1, 4);                            \
  else if (ks == 2) NXD_GV(MMV, 2, 4);                       \
  else if (p.K <= 8192) NXD_GV(MMV, 4, 4);                   \
  else NXD_GV(MMV, 4, 6)
  if (p.M == 1) { NXD_GV_KS(1); }
  else if (p.M == 2) { NXD_GV_KS(2); }
  else if (ks == 1) NXD_GV(4, 1, 4);
  else if (ks == 2) NXD_GV(4, 2, 4);
  else NXD_GV(4, 4, 4);
#undef NXD_GV_KS
#undef NXD_GV
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

template <int EPI>
static int run_rows(const GemvHyperParams& p, hipStream_t s) {
  if constexpr (EPI != HYPER)
    if (p.u) return run_gemv<true, EPI>(p, s);
  return run_gemv<false, EPI>(p, s);
}

}  // namespace hybrid

int gemv_hyper_launch(int epi, const GemvHyperParams& p, hipStream_t s) {
  using namespace hybrid;
  switch (epi) {
    case STORE: return run_rows<STORE>(p, s);
    case RELU2: return run_rows<RELU2>(p, s);
    case F32CAP: return run_rows<F32CAP>(p, s);
    case HYPER: return run_rows<HYPER>(p, s);
  }
  return -1;
}

}  // namespace nxd
