// Generalised delta rule (a linear-attention recurrence with a matrix state per head, decay and removal
// per key channel), token by token:
//
//   S <- diag(w) S - (a u) (u^T S) + k v^T   (both terms read the old state);  o = S^T r
//   u = k / sqrt(sum k^2 + 1e-6),  w = exp(-e^(-1/2) sigmoid(W2 tanh(low) + w0)),  a = sigmoid(. + bias)
//   y = out_scale * o / rms(o) * norm_w * sigmoid(gate)                       (rms per head)
//
// Everything after the projections is fp32.  The state of a sequence lives in the cache as
// [slot][H][D (value)][DP (key)], the padding stays zero; a sequence's first token starts from zero, so a
// slot needs no clearing.
//
// One workgroup a (head, sequence), whose state columns stay in its registers over all tokens of the step:
// 8 lanes a column.  Long runs of tokens: channel_delta_chunk.hip.
#include "channel_delta.h"

namespace nxd {
namespace hybrid {

// 8 elements of a row of W2 (16-byte aligned rows) times 8 of LDS
__device__ __forceinline__ float dot8_lds(const uint16_t* w, const float* x) {
  float f[8], s = 0.f;
  unpack8(*reinterpret_cast<const u32x4_t*>(w), f);
#pragma unroll
  for (int i = 0; i < 8; ++i) s += f[i] * x[i];
  return s;
}
__device__ __forceinline__ float dot8_lds(const float* w, const float* x) {
  const f32x4_t a = ld4(w), b = ld4(w + 4);
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) s += a[i] * x[i] + b[i] * x[4 + i];
  return s;
}

template <typename T, int NI, int NTH>
__global__ void __launch_bounds__(NTH) channel_delta_step_kernel(ChannelDeltaParams p) {
  constexpr int DP = NI * 32, COLS = NTH / 8, PASS = (DP + COLS - 1) / COLS;
  extern __shared__ __attribute__((aligned(16))) float low[];   // [N]
  __shared__ __attribute__((aligned(16))) float us[DP], ks[DP], rs[DP], ws[DP], bs[DP];
  __shared__ float vs[DP], os[DP], red[16], red2[16];
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, l = tid & 7, col = tid >> 3;
  const int h = blockIdx.x, b = blockIdx.y, H = p.H, D = p.D, N = p.N, HD = H * D;
  const int slot = slot_of(p.slots, b, p.nslots);
  const int64_t p0 = pos_of(p.pos, p.pos_stride, b);
  const int len = p.lens ? min(max(p.lens[b], 0), p.T) : p.T;
  const bool wide = N % 8 == 0;   // rows of W2 in 16-byte pieces
  float* state = p.state + ((int64_t)slot * H + h) * D * DP;
  f32x4_t S[PASS][NI];
#pragma unroll
  for (int q = 0; q < PASS; ++q)
#pragma unroll
    for (int i = 0; i < NI; ++i)
      S[q][i] = p0 > 0 ? ld4(state + (int64_t)min(col + q * COLS, D - 1) * DP + i * 32 + l * 4) : f32x4_t{0.f, 0.f, 0.f, 0.f};
  T* yb = static_cast<T*>(p.y) + (int64_t)b * p.T * p.ldy + h * D;
  for (int t = 0; t < len; ++t) {
    const T* row = static_cast<const T*>(p.proj) + ((int64_t)b * p.T + t) * p.ldp + h * D;
    if (t > 0) __syncthreads();   // the last token's readers of LDS are done
    float sk = 0.f;
    for (int d = tid; d < DP; d += NTH) {
      const bool in = d < D;
      const float k = in ? ld(row + HD + d) : 0.f;
      ks[d] = k;
      rs[d] = in ? ld(row + d) : 0.f;
      vs[d] = in ? ld(row + 2 * HD + d) : 0.f;
      bs[d] = in ? 1.f / (1.f + expf(-(ld(row + 4 * HD + d) + p.a_bias[h * D + d]))) : 0.f;
      sk += k * k;
    }
    for (int j = tid; j < N; j += NTH) low[j] = tanhf_(ld(row + 5 * HD - h * D + j));
    sk = sum64(sk);
    if (lane == 0) red[wid] = sk;
    __syncthreads();
    sk = 0.f;
#pragma unroll
    for (int i = 0; i < NTH / 64; ++i) sk += red[i];
    const float rn = 1.f / sqrtf(sk + 1e-6f);
    for (int c0 = 0; c0 < DP; c0 += NTH / 4) {   // four lanes a channel
      const int c = c0 + tid / 4;
      const bool in = c < D;
      const T* w = static_cast<const T*>(p.w2) + (int64_t)(h * D + min(c, D - 1)) * N;
      float x = 0.f;
      if (wide) {
        for (int j = (tid & 3) * 8; j < N; j += 32) x += dot8_lds(w + j, low + j);
      } else {
        for (int j = tid & 3; j < N; j += 4) x += ld(w + j) * low[j];
      }
      x = sum_lanes<4>(x);
      if ((tid & 3) == 0 && c < DP) {
        const float u = ks[c] * rn;
        us[c] = u;
        ws[c] = in ? __builtin_amdgcn_exp2f(decay_log2(x + p.w0[h * D + c])) : 0.f;
        bs[c] *= u;
      }
    }
    __syncthreads();
    f32x4_t u[NI], w[NI], a[NI], k[NI], r[NI];
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int o = i * 32 + l * 4;
      u[i] = ld4(us + o);
      w[i] = ld4(ws + o);
      a[i] = ld4(bs + o);
      k[i] = ld4(ks + o);
      r[i] = ld4(rs + o);
    }
    float so = 0.f;
#pragma unroll
    for (int q = 0; q < PASS; ++q) {
      const int v = col + q * COLS;
      float z = 0.f, out = 0.f;
#pragma unroll
      for (int i = 0; i < NI; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) z += S[q][i][e] * u[i][e];
      z = sum8(z);
      const float x = v < D ? vs[v] : 0.f;
#pragma unroll
      for (int i = 0; i < NI; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          S[q][i][e] = S[q][i][e] * w[i][e] - a[i][e] * z + k[i][e] * x;
          out += S[q][i][e] * r[i][e];
        }
      out = sum8(out);
      if (l == 0 && v < D) {
        os[v] = out;
        so += out * out;
      }
    }
    so = sum64(so);
    if (lane == 0) red2[wid] = so;
    __syncthreads();
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NTH / 64; ++i) ss += red2[i];
    const float f = p.out_scale / sqrtf(ss / (float)D + p.eps);
    for (int v = tid; v < D; v += NTH)
      st(yb + (int64_t)t * p.ldy + v, os[v] * f * p.norm_w[h * D + v] * sigmoidf_(ld(row + 3 * HD + v)));
  }
  if (len > 0) {
#pragma unroll
    for (int q = 0; q < PASS; ++q)
      if (col + q * COLS < D) {
#pragma unroll
        for (int i = 0; i < NI; ++i) st4(state + (int64_t)(col + q * COLS) * DP + i * 32 + l * 4, S[q][i]);
      }
  }
  for (int t = len; t < p.T; ++t)   // padding: a defined value for the projection
    for (int v = tid; v < D; v += NTH) st(yb + (int64_t)t * p.ldy + v, 0.f);
}

template <typename T>
static int run_step(const ChannelDeltaParams& p, hipStream_t s) {
  const dim3 grid((unsigned)p.H, (unsigned)p.B);
  const size_t lds = (size_t)p.N * 4;
#define NXD_STEP(NI, NTH) hipLaunchKernelGGL((channel_delta_step_kernel<T, NI, NTH>), grid, dim3(NTH), lds, s, p)
  switch (p.DP / 32) {
    case 1: NXD_STEP(1, 256); break;
    case 2: NXD_STEP(2, 256); break;
    case 3: NXD_STEP(3, 512); break;
    case 4: NXD_STEP(4, 512); break;
    case 5: NXD_STEP(5, 1024); break;
    case 6: NXD_STEP(6, 1024); break;
    case 7: NXD_STEP(7, 1024); break;
    case 8: NXD_STEP(8, 1024); break;
    default: return -1;
  }
#undef NXD_STEP
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

}  // namespace hybrid

int channel_delta_step_launch(bool f32, const ChannelDeltaParams& p, hipStream_t s) {
  return f32 ? hybrid::run_step<float>(p, s) : hybrid::run_step<uint16_t>(p, s);
}

}  // namespace nxd
