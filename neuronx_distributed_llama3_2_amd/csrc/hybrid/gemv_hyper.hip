// Decode projections (1 to 16 rows) of hyper-connected decoders, with the element-wise work around them:
//
//   NORM prologue : x = rms_normalise(u) (1 + norm_w) from the fp32 sublayer input u [M, K]
//   epilogues     : store (bf16) | squared ReLU (bf16) | fp32 with an optional cap tanh(y / cap)
//                   | HYPER: y + bias goes straight into the residual streams, x_t = sum_s mix[s][t] x_s +
//                   write[t] y, and u = sum_t read[t] x_t of the next sublayer comes out -- a column of
//                   the streams belongs to the one wave that owns the weight row, so it is updated in place
//
// So a sublayer is three launches: norm + projection, mixer (or nothing), projection + streams.
//
// Decode streams every weight byte once.  Up to 2 rows: a wave per weight row (or a K slice of it), bf16
// dot products, a round of weight loads in flight before the prologue runs.  3 to 16 rows:
// v_mfma_f32_16x16x32_bf16 with 16 weight rows as the B operand and the activations as A.
#include "gemv_hyper.h"

namespace nxd {

namespace hybrid {

enum GemvEpi { STORE = 0, RELU2 = 1, F32CAP = 2, HYPER = 3 };

// one output value of row m, column n
template <int EPI>
__device__ __forceinline__ void emit(const GemvHyperParams& p, int m, int n, float v) {
  if (EPI == STORE) {
    static_cast<uint16_t*>(p.y)[(int64_t)m * p.ldy + n] = f2bf(v);
  } else if (EPI == RELU2) {
    const float r = fmaxf(v, 0.f);
    static_cast<uint16_t*>(p.y)[(int64_t)m * p.ldy + n] = f2bf(r * r);
  } else if (EPI == F32CAP) {
    static_cast<float*>(p.y)[(int64_t)m * p.ldy + n] = p.cap > 0.f ? p.cap * tanhf(v / p.cap) : v;
  } else {
    v = bf2f(f2bf(v)) + (p.bias ? p.bias[n] : 0.f);   // the projection's output is a bf16 activation
    float* x = p.streams + (int64_t)m * p.S * p.N + n;
    float old[8], u = 0.f;
#pragma unroll
    for (int s = 0; s < 8; ++s) old[s] = s < p.S ? x[(int64_t)s * p.N] : 0.f;
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
template <int MM, bool NORM, int EPI, int KS>
__global__ void __launch_bounds__(256) gemv_hyper_kernel(GemvHyperParams p) {
  constexpr int U = 4;   // 512-element steps of a load round
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
  u32x4_t wv[U];
  auto load_round = [&](int base) {   // lanes past the end read the slice's last piece and skip it below
#pragma unroll
    for (int i = 0; i < U; ++i)
      wv[i] = __builtin_nontemporal_load(reinterpret_cast<const u32x4_t*>(wrow + min(base + i * 512 + lane * 8, kend - 8)));
  };
  load_round(kbeg);
  if constexpr (NORM) norm_rows<MM, 256>(p, xs, red, first);
  float acc[MM];
#pragma unroll
  for (int m = 0; m < MM; ++m) acc[m] = 0.f;
  for (int base = kbeg; some && base < kend; base += 512 * U) {
    if (base != kbeg) load_round(base);
#pragma unroll
    for (int i = 0; i < U; ++i) {
      const int k = base + i * 512 + lane * 8;
      if (k < kend) {
#pragma unroll
        for (int m = 0; m < MM; ++m)
          if (m < p.M)
            acc[m] = dot8_bf16(*reinterpret_cast<const u32x4_t*>(NORM ? xs + m * p.K + k : p.x + (int64_t)m * p.ldx + k), wv[i], acc[m]);
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
  if constexpr (MM == 2) v = lane == 1 ? acc[1] : v;
  emit<EPI>(p, lane, n, v);   // lane m: row m
}

// ---- 3 to 16 rows on the matrix cores.  A wave owns 16 weight rows (or a K slice of them).
template <bool NORM, int EPI, int KS, int NWV>
__global__ void __launch_bounds__(64 * NWV) gemm16_hyper_kernel(GemvHyperParams p) {
  constexpr int U = 4, MM = 16;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  uint16_t* xs = reinterpret_cast<uint16_t*>(smem);
  __shared__ float red[NWV][MM];
  __shared__ f32x4_t part[KS > 1 ? NWV : 1][64];
  const int tid = threadIdx.x, lane = tid & 63, wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int tile = blockIdx.x * (NWV / KS) + wid / KS, ks = wid % KS, c = lane & 15, kq = 8 * (lane >> 4);
  const uint16_t* wrow = p.w + (int64_t)min(tile * 16 + c, p.N - 1) * p.ldw;
  const int kc = ((p.K + KS - 1) / KS + 31) & ~31;
  const int kbeg = min(ks * kc, p.K), kend = min(p.K, kbeg + kc);
  u32x4_t wv[2][U];
  auto load_w = [&](u32x4_t (&d)[U], int base) {
#pragma unroll
    for (int i = 0; i < U; ++i)
      d[i] = __builtin_nontemporal_load(reinterpret_cast<const u32x4_t*>(wrow + min(base + 32 * i + kq, p.K - 8)));
  };
  load_w(wv[0], kbeg);
  load_w(wv[1], kbeg + 32 * U);
  if constexpr (NORM) {
    constexpr int NT = 64 * NWV;
    float ss[MM];
#pragma unroll
    for (int m = 0; m < MM; ++m) {
      ss[m] = 0.f;
      if (m < p.M)
        for (int k = tid * 4; k < p.K; k += NT * 4) {
          const f32x4_t a = ld4(p.u + (int64_t)m * p.K + k);
#pragma unroll
          for (int i = 0; i < 4; ++i) ss[m] += a[i] * a[i];
        }
    }
#pragma unroll
    for (int m = 0; m < MM; ++m) {
      const float s = sum64(ss[m]);
      if (lane == 0) red[wid][m] = s;
    }
    __syncthreads();
#pragma unroll
    for (int m = 0; m < MM; ++m) {
      if (m < p.M) {
        float t = 0.f;
#pragma unroll
        for (int i = 0; i < NWV; ++i) t += red[i][m];
        const float rstd = 1.f / sqrtf(t / (float)p.K + p.eps);
        for (int k = tid * 4; k < p.K; k += NT * 4) {
          const f32x4_t a = ld4(p.u + (int64_t)m * p.K + k), gw = ld4(p.norm_w + k);
          st4(xs + m * p.K + k, f32x4_t{a[0] * rstd * (1.f + gw[0]), a[1] * rstd * (1.f + gw[1]), a[2] * rstd * (1.f + gw[2]),
                                        a[3] * rstd * (1.f + gw[3])});
        }
      }
    }
    __syncthreads();
  }
  const uint16_t* xr = NORM ? xs + min(c, p.M - 1) * p.K : p.x + (int64_t)min(c, p.M - 1) * p.ldx;
  f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
  auto round = [&](const u32x4_t (&wr)[U], int base) {
    u32x4_t xa[U];
#pragma unroll
    for (int i = 0; i < U; ++i) {   // rows and columns past the end: an in-bounds piece replaced by zeros
      const int k = base + 32 * i + kq;
      const u32x4_t v = *reinterpret_cast<const u32x4_t*>(xr + min(k, p.K - 8));
      xa[i] = c < p.M && k < kend ? v : u32x4_t{0u, 0u, 0u, 0u};
    }
#pragma unroll
    for (int i = 0; i < U; ++i)
      if (base + 32 * i < kend)
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, xa[i]), __builtin_bit_cast(bf16x8_t, wr[i]), acc, 0, 0, 0);
  };
#pragma unroll 1
  for (int base = kbeg; base < kend; base += 64 * U) {
    round(wv[0], base);
    load_w(wv[0], base + 64 * U);
    round(wv[1], base + 32 * U);
    load_w(wv[1], base + 96 * U);
  }
  if constexpr (KS > 1) {
    part[wid][lane] = acc;
    __syncthreads();
    if (ks != 0) return;
#pragma unroll
    for (int i = 1; i < KS; ++i) acc += part[wid + i][lane];
  }
  const int n = tile * 16 + c, m0 = 4 * (lane >> 4);
  if (n >= p.N) return;
#pragma unroll
  for (int i = 0; i < 4; ++i)
    if (m0 + i < p.M) emit<EPI>(p, m0 + i, n, acc[i]);
}

template <bool NORM, int EPI>
static int run_gemv(const GemvHyperParams& p, hipStream_t s) {
  const size_t lds = NORM ? (size_t)p.M * p.K * 2 : 0;
  if (p.M <= 2) {
    // K slices while the grid stays below 8,192 waves and a slice keeps 1,024 elements
    int ks = 1;
    while (ks < 4 && (int64_t)p.N * ks * 2 <= 8192 && p.K / (ks * 2) >= 1024) ks *= 2;
    const dim3 grid((unsigned)((p.N * ks + 3) / 4)), block(256);
#define NXD_GV(MMV, KSV) hipLaunchKernelGGL((gemv_hyper_kernel<MMV, NORM, EPI, KSV>), grid, block, lds, s, p)
    if (p.M == 1) { if (ks == 1) NXD_GV(1, 1); else if (ks == 2) NXD_GV(1, 2); else NXD_GV(1, 4); }
    else { if (ks == 1) NXD_GV(2, 1); else if (ks == 2) NXD_GV(2, 2); else NXD_GV(2, 4); }
#undef NXD_GV
    return hipGetLastError() == hipSuccess ? 0 : 1;
  }
  const int tiles = (p.N + 15) / 16;
  int ks = 1;
  while (ks < 8 && (int64_t)tiles * ks < 2048 && p.K / (ks * 2) >= 256) ks *= 2;
#define NXD_GM(KSV, NW) hipLaunchKernelGGL((gemm16_hyper_kernel<NORM, EPI, KSV, NW>), dim3((unsigned)ceil_div(tiles, NW / KSV)), dim3(64 * NW), lds, s, p)
  if (ks == 8) NXD_GM(8, 8);
  else if (ks == 4) NXD_GM(4, 4);
  else if (ks == 2) NXD_GM(2, 4);
  else NXD_GM(1, 4);
#undef NXD_GM
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

}  // namespace hybrid

int gemv_hyper_launch(int epi, bool norm, const GemvHyperParams& p, hipStream_t s) {
  using namespace hybrid;
  switch (epi) {
    case STORE: return norm ? run_gemv<true, STORE>(p, s) : run_gemv<false, STORE>(p, s);
    case RELU2: return norm ? run_gemv<true, RELU2>(p, s) : run_gemv<false, RELU2>(p, s);
    case F32CAP: return norm ? run_gemv<true, F32CAP>(p, s) : run_gemv<false, F32CAP>(p, s);
    case HYPER: return norm ? -1 : run_gemv<false, HYPER>(p, s);
  }
  return -1;
}

}  // namespace nxd
