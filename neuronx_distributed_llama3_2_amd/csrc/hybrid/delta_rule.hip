// Gated delta rule (a linear-attention recurrence with a matrix state per head):
//
//   q, k, v <- silu(causal conv of the projections); q, k unit vectors per head (q also * D^-1/2)
//   S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//   y = o / rms(o) * norm_w * silu(gate)                        (per head, over its V values)
//
// Everything here after the projections is computed in fp32.  The state of a sequence lives in the
// cache: S as [slot][H][V][DP] fp32 (DP = D rounded up to 32, the padding stays zero), and the
// convolution's inputs as a ring [slot][taps][C] in the activation type, position p in entry p % taps.
// Whether a token has a predecessor is decided by its position, so a slot needs no clearing before it
// is used again.  The projection buffer's columns are [q (G D) | k (G D) | v (H V) | gate (H V) |
// beta (H) | decay (H)].
//
//   delta_prep   : convolution, silu, unit norms, gates of all tokens of a step
//   delta_scan   : the recurrence, token by token, from the cached state (8 lanes a state column)
//                  (long runs of tokens: 64 at a time, delta_chunk.hip)
//   delta_out    : the gated head norm
//   delta_decode : all of it for one new token per sequence, one workgroup per (sequence, head)
#include "hybrid.h"
#include "delta_rule.h"

namespace nxd {
namespace hybrid {

// convolution + silu of one channel for the token of row m (position ps): earlier tokens of this
// step come from the projection buffer, older ones from the ring
template <typename T>
__device__ __forceinline__ float conv_silu(const DeltaParams& p, const T* proj, const T* ring, int64_t m, int t,
                                           int64_t ps, int c) {
  const int C = p.C, n = p.taps;
  float a = 0.f;
  for (int j = 0; j < n; ++j) {
    const int back = n - 1 - j;
    const int64_t q = ps - back;
    if (q < 0) continue;
    const float x = back <= t ? ld(proj + (m - back) * p.ldp + c) : ld(ring + (q % n) * C + c);
    a += p.conv[(int64_t)j * C + c] * x;
  }
  return siluf_(a);
}

// the same with every load of up to 4 taps issued at once
template <typename T>
__device__ __forceinline__ float conv_silu4(const DeltaParams& p, const T* row, const T* ring, int64_t ps, int c) {
  float a = p.conv[(int64_t)(p.taps - 1) * p.C + c] * ld(row + c);
#pragma unroll
  for (int back = 1; back < 4; ++back) {
    const int64_t q = ps - back;
    const bool in = back < p.taps && q >= 0;
    const int e = in ? (int)(q % p.taps) : 0, j = in ? p.taps - 1 - back : 0;
    const float x = ld(ring + (int64_t)e * p.C + c), w = p.conv[(int64_t)j * p.C + c];
    a += in ? x * w : 0.f;
  }
  return siluf_(a);
}

// the same for TT consecutive tokens t0 .. of sequence b and N neighbouring channels c ..: every input is
// read once (up to 4 taps; more fall back to the single-token form)
template <typename T, int TT, int N>
__device__ __forceinline__ void conv_silu_run(const DeltaParams& p, const T* proj, const T* ring, int64_t m0, int t0, int n,
                                              int64_t p0, int c, float (&out)[N][TT]) {
  if (p.taps > 4) {
#pragma unroll
    for (int k = 0; k < N; ++k)
#pragma unroll
      for (int i = 0; i < TT; ++i) out[k][i] = i < n ? conv_silu<T>(p, proj, ring, m0 + i, t0 + i, p0 + i, c + k) : 0.f;
    return;
  }
  float x[N][TT + 3], wt[N][4];
#pragma unroll
  for (int j = 0; j < 4; ++j)
#pragma unroll
    for (int k = 0; k < N; ++k) wt[k][j] = j < 4 - p.taps ? 0.f : p.conv[(int64_t)(j - 4 + p.taps) * p.C + c + k];
  auto get = [&](const T* s, int i) {
    if constexpr (N == 2) ld2(s, x[0][i], x[1][i]);
    else x[0][i] = ld(s);
  };
  if (t0 >= 3 && n == TT) {   // (uniform) no edge of the sequence or of the step in sight
#pragma unroll
    for (int i = 0; i < TT + 3; ++i) get(proj + (m0 + i - 3) * p.ldp + c, i);
  } else {
#pragma unroll
    for (int i = 0; i < TT + 3; ++i) {   // token t0 + i - 3
      const int64_t q = p0 + i - 3;
#pragma unroll
      for (int k = 0; k < N; ++k) x[k][i] = 0.f;
      if (i - 3 < n && q >= 0 && 3 - i < p.taps) get(t0 + i - 3 >= 0 ? proj + (m0 + i - 3) * p.ldp + c : ring + (q % p.taps) * p.C + c, i);
    }
  }
#pragma unroll
  for (int k = 0; k < N; ++k)
#pragma unroll
    for (int i = 0; i < TT; ++i)
      out[k][i] = siluf_(wt[k][0] * x[k][i] + wt[k][1] * x[k][i + 1] + wt[k][2] * x[k][i + 2] + wt[k][3] * x[k][i + 3]);
}

constexpr int PREP_TOKENS = 8;   // tokens of one sequence a prep workgroup handles

// N = 2: two neighbouring channels a lane (even head sizes), 1: one.  NJ steps of 64 N columns cover DP.
template <typename T, int N, int NJ>
__global__ void __launch_bounds__(256) delta_prep_kernel(DeltaParams p) {
  constexpr int TT = PREP_TOKENS;
  const int b = blockIdx.y, t0 = blockIdx.x * TT;
  const int len = p.lens ? min(p.lens[b], p.T) : p.T;
  const bool frag = p.nch > 0;
  // the chunked scan reads whole chunks: their last tokens past the sequence are zeros
  if (t0 >= (frag ? (len + 63) / 64 * 64 : len)) return;
  const int n = max(0, min(TT, len - t0));
  const int64_t m0 = (int64_t)b * p.T + t0;
  const int64_t p0 = pos_of(p.pos, p.pos_stride, b) + t0;
  const int slot = slot_of(p.slots, b, p.nslots);
  const T* proj = static_cast<const T*>(p.proj);
  const T* ring = static_cast<const T*>(p.ring) + (int64_t)slot * p.taps * p.C;
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int G = p.G, D = p.D, DP = p.DP, H = p.H, HV = p.H * p.V, NB = DP / 16;
  for (int hd = wid; hd < 2 * G; hd += 4) {   // q heads, then k heads: a wave per unit vector
    const bool isq = hd < G;
    const int g = isq ? hd : hd - G;
    float x[NJ][N][TT], ss[TT];
#pragma unroll
    for (int i = 0; i < TT; ++i) ss[i] = 0.f;
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
      const int d = N * lane + 64 * N * j;
#pragma unroll
      for (int k = 0; k < N; ++k)
#pragma unroll
        for (int i = 0; i < TT; ++i) x[j][k][i] = 0.f;
      if (d < D && n > 0) conv_silu_run<T, TT, N>(p, proj, ring, m0, t0, n, p0, hd * D + d, x[j]);
#pragma unroll
      for (int k = 0; k < N; ++k)
#pragma unroll
        for (int i = 0; i < TT; ++i) ss[i] += x[j][k][i] * x[j][k][i];
    }
#pragma unroll
    for (int i = 0; i < TT; ++i) {
      float r = __builtin_amdgcn_rsqf(sum64(ss[i]) + 1e-6f);
      if (isq) r *= p.qscale;
      if (i >= n) r = 0.f;
#pragma unroll
      for (int j = 0; j < NJ; ++j)
#pragma unroll
        for (int k = 0; k < N; ++k) x[j][k][i] *= r;
    }
    if (!frag) {
      float* out = (isq ? p.qn : p.kn) + (m0 * G + g) * DP;
#pragma unroll
      for (int j = 0; j < NJ; ++j)
#pragma unroll
        for (int k = 0; k < N; ++k) {
          const int d = N * lane + 64 * N * j + k;
#pragma unroll
          for (int i = 0; i < TT; ++i)
            if (i < n && d < DP) out[(int64_t)i * G * DP + d] = x[j][k][i];
        }
      continue;
    }
    // fragment order of the chunk (delta_chunk.hip): q as rows of tokens, k as rows of columns
    const int tc = t0 & 63, tb = tc >> 4;
    const int64_t cell = (((int64_t)b * p.nch + t0 / 64) * G + g) * 64 * DP;
    if constexpr (N == 2) {
      if (isq) {   // neighbouring lanes swap halves: four channels of four tokens each, 16 bytes a token
        const bool odd = lane & 1;
#pragma unroll
        for (int j = 0; j < NJ; ++j) {
          const int d = (2 * lane + 128 * j) & ~3;
          float* out = p.qn + cell + ((((int64_t)tb * NB + d / 16) * 4 + (d & 15) / 4) * 16 + (tc & 15) + (odd ? 4 : 0)) * 4;
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            float mine[2], other[2];
#pragma unroll
            for (int k = 0; k < 2; ++k) {
              const float send = odd ? x[j][k][i] : x[j][k][4 + i];
              other[k] = __uint_as_float(__builtin_amdgcn_update_dpp(0, __float_as_uint(send), 0xB1, 0xf, 0xf, true));
              mine[k] = odd ? x[j][k][4 + i] : x[j][k][i];
            }
            if (d < DP)
              st4(out + 4 * i, odd ? f32x4_t{other[0], other[1], mine[0], mine[1]} : f32x4_t{mine[0], mine[1], other[0], other[1]});
          }
        }
        continue;
      }
    }
#pragma unroll
    for (int j = 0; j < NJ; ++j)
#pragma unroll
      for (int k = 0; k < N; ++k) {
        const int d = N * lane + 64 * N * j + k;
        if (d >= DP) continue;
        if (isq) {
          float* out = p.qn + cell + ((((int64_t)tb * NB + d / 16) * 4 + (d & 15) / 4) * 16 + (tc & 15)) * 4 + (d & 3);
#pragma unroll
          for (int i = 0; i < TT; ++i) out[4 * i] = x[j][k][i];
        } else {
          float* out = p.kn + cell + ((((int64_t)(d / 16) * 4 + tb) * 4 + (tc & 15) / 4) * 16 + (d & 15)) * 4;
          st4(out, f32x4_t{x[j][k][0], x[j][k][1], x[j][k][2], x[j][k][3]});
          st4(out + 64, f32x4_t{x[j][k][4], x[j][k][5], x[j][k][6], x[j][k][7]});
        }
      }
  }
  if (n <= 0) return;
  float* vo = p.vn + m0 * HV;
  for (int c = N * tid; c < HV; c += 256 * N) {
    float x[N][TT];
    conv_silu_run<T, TT, N>(p, proj, ring, m0, t0, n, p0, 2 * G * D + c, x);
#pragma unroll
    for (int i = 0; i < TT; ++i)
      if (i < n) {
        if constexpr (N == 2) *reinterpret_cast<float2*>(vo + (int64_t)i * HV + c) = float2{x[0][i], x[1][i]};
        else vo[(int64_t)i * HV + c] = x[0][i];
      }
  }
  for (int i = tid; i < n * H; i += 256) {
    const int h = i % H;
    const int64_t m = m0 + i / H;
    const T* gates = proj + m * p.ldp + p.C + HV;
    p.beta[m * H + h] = sigmoidf_(ld(gates + h));
    p.lg[m * H + h] = -expf(p.a_log[h]) * softplusf_(ld(gates + H + h) + p.dt_bias[h]);
  }
}

// ---- the recurrence, one token after another.  A workgroup owns 32 columns of one head's state
// (8 lanes a column, NI float4 of the column's DP entries each).
template <typename T, int NI>
__global__ void __launch_bounds__(256) delta_scan_kernel(DeltaParams p) {
  constexpr int TK = 16, DP = NI * 32;
  __shared__ __attribute__((aligned(16))) float ks[TK][DP], qs[TK][DP];
  __shared__ float vs[TK][32], gs[TK], bs[TK];
  const int tid = threadIdx.x, l = tid & 7, col = tid >> 3;
  const int h = blockIdx.y, b = blockIdx.z, v = blockIdx.x * 32 + col;
  const int H = p.H, G = p.G, V = p.V, g = h / (H / G);
  const int len = p.lens ? min(p.lens[b], p.T) : p.T;
  if (len <= 0) return;
  const int slot = slot_of(p.slots, b, p.nslots);
  const int64_t p0 = pos_of(p.pos, p.pos_stride, b);
  float* state = p.state + (((int64_t)slot * H + h) * V + min(v, V - 1)) * DP;
  f32x4_t S[NI];
#pragma unroll
  for (int i = 0; i < NI; ++i) S[i] = p0 > 0 ? ld4(state + i * 32 + l * 4) : f32x4_t{0.f, 0.f, 0.f, 0.f};
  const int64_t m0 = (int64_t)b * p.T;
  for (int t0 = 0; t0 < len; t0 += TK) {
    const int n = min(TK, len - t0);
    __syncthreads();
    for (int i = tid; i < n * DP; i += 256) {
      const int t = i / DP, d = i % DP;
      const int64_t o = ((m0 + t0 + t) * G + g) * DP + d;
      ks[t][d] = p.kn[o];
      qs[t][d] = p.qn[o];
    }
    for (int i = tid; i < n * 32; i += 256) {
      const int t = i >> 5, c = blockIdx.x * 32 + (i & 31);
      vs[t][i & 31] = c < V ? p.vn[((m0 + t0 + t) * H + h) * V + c] : 0.f;
    }
    if (tid < n) {
      gs[tid] = expf(p.lg[(m0 + t0 + tid) * H + h]);
      bs[tid] = p.beta[(m0 + t0 + tid) * H + h];
    }
    __syncthreads();
    for (int t = 0; t < n; ++t) {
      const float gt = gs[t];
      f32x4_t k[NI];
      float dot = 0.f;
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        k[i] = ld4(&ks[t][i * 32 + l * 4]);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          S[i][e] *= gt;
          dot += S[i][e] * k[i][e];
        }
      }
      dot = sum8(dot);
      const float u = bs[t] * (vs[t][col] - dot);
      float out = 0.f;
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        const f32x4_t q = ld4(&qs[t][i * 32 + l * 4]);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          S[i][e] += k[i][e] * u;
          out += S[i][e] * q[e];
        }
      }
      out = sum8(out);
      if (l == 0 && v < V) p.o[((m0 + t0 + t) * H + h) * V + v] = out;
    }
  }
  if (v < V) {
#pragma unroll
    for (int i = 0; i < NI; ++i) st4(state + i * 32 + l * 4, S[i]);
  }
  if (blockIdx.x == 0 && h == 0) ring_write<T>(p, b, slot, p0, len, tid, 256);
}

template <typename T>
__global__ void __launch_bounds__(256) delta_out_kernel(DeltaParams p) {
  const int lane = threadIdx.x & 63;
  const int64_t i = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);   // (row, head)
  const int H = p.H, V = p.V;
  if (i >= (int64_t)p.B * p.T * H) return;
  const int64_t m = i / H;
  const int h = (int)(i % H);
  T* y = static_cast<T*>(p.y) + m * p.ldy + h * V;
  if (p.lens && (int)(m % p.T) >= p.lens[m / p.T]) {   // padding: a defined value for the projection
    for (int v = lane; v < V; v += 64) st(y + v, 0.f);
    return;
  }
  const float* o = p.o + i * V;
  const T* gate = static_cast<const T*>(p.proj) + m * p.ldp + p.C + h * V;
  float x[4], ss = 0.f;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int v = lane + 64 * j;
    x[j] = v < V ? o[v] : 0.f;
    ss += x[j] * x[j];
  }
  const float r = 1.f / sqrtf(sum64(ss) / (float)V + p.eps);
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int v = lane + 64 * j;
    if (v < V) st(y + v, x[j] * r * p.norm_w[v] * siluf_(ld(gate + v)));
  }
}

// The same for V a multiple of 4: four values a lane, L lanes a head.
template <typename T, int L>
__global__ void __launch_bounds__(256) delta_out4_kernel(DeltaParams p) {
  const int64_t i = (int64_t)blockIdx.x * (256 / L) + threadIdx.x / L;   // (row, head)
  const int H = p.H, V = p.V, v = (threadIdx.x % L) * 4;
  const bool in = i < (int64_t)p.B * p.T * H && v < V;
  const int64_t m = in ? i / H : 0;
  const int h = in ? (int)(i % H) : 0;
  const bool live = in && !(p.lens && (int)(m % p.T) >= p.lens[m / p.T]);
  f32x4_t x = {0.f, 0.f, 0.f, 0.f}, g = x, w = x;
  if (live) {
    x = ld4(p.o + i * V + v);
    g = ld4(static_cast<const T*>(p.proj) + m * p.ldp + p.C + h * V + v);
    w = ld4(p.norm_w + v);
  }
  const float ss = sum_lanes<L>(x[0] * x[0] + x[1] * x[1] + x[2] * x[2] + x[3] * x[3]);
  if (!in) return;
  const float r = 1.f / sqrtf(ss / (float)V + p.eps);
#pragma unroll
  for (int j = 0; j < 4; ++j) x[j] *= r * w[j] * siluf_(g[j]);   // padding: zeros
  st4(static_cast<T*>(p.y) + m * p.ldy + h * V + v, x);
}

// ---- one new token per sequence: a workgroup of NTH threads per (head, sequence)
template <typename T, int NI, int NTH>
__global__ void __launch_bounds__(NTH) delta_decode_kernel(DeltaParams p) {
  constexpr int DP = NI * 32, COLS = NTH / 8;
  __shared__ __attribute__((aligned(16))) float qs[DP], ks[DP];
  __shared__ float vs[256], os[256], red[16], red2[16], red3[16];
  const int tid = threadIdx.x, l = tid & 7, col = tid >> 3;
  const int h = blockIdx.x, b = blockIdx.y;
  const int H = p.H, G = p.G, D = p.D, V = p.V, rep = H / G, g = h / rep, C = p.C;
  const int slot = slot_of(p.slots, b, p.nslots);
  const int64_t ps = pos_of(p.pos, p.pos_stride, b);
  const T* proj = static_cast<const T*>(p.proj);
  T* ring = static_cast<T*>(p.ring) + (int64_t)slot * p.taps * C;
  float* state = p.state + ((int64_t)slot * H + h) * V * DP;
  // the first columns of the state are on their way while the inputs are prepared
  f32x4_t S[NI];
  {
    const float* sp = state + (int64_t)min(col, V - 1) * DP;
#pragma unroll
    for (int i = 0; i < NI; ++i) S[i] = ld4(sp + i * 32 + l * 4);
  }
  T* entry = ring + (ps % p.taps) * C;   // this token's ring entry: read by nobody in this launch
  float sq = 0.f, sk = 0.f;
  for (int i = tid; i < 2 * DP + V; i += NTH) {
    const int part = i < DP ? 0 : (i < 2 * DP ? 1 : 2);
    const int d = part == 0 ? i : (part == 1 ? i - DP : i - 2 * DP);
    float x = 0.f;
    if (part == 2 || d < D) {
      const int c = part == 0 ? g * D + d : (part == 1 ? (G + g) * D + d : 2 * G * D + h * V + d);
      x = p.taps <= 4 ? conv_silu4<T>(p, proj + (int64_t)b * p.ldp, ring, ps, c) : conv_silu<T>(p, proj, ring, b, 0, ps, c);
      if (part == 2 || h % rep == 0) entry[c] = proj[(int64_t)b * p.ldp + c];
    }
    if (part == 0) { qs[d] = x; sq += x * x; }
    else if (part == 1) { ks[d] = x; sk += x * x; }
    else vs[d] = x;
  }
  const int lane = tid & 63, wid = tid >> 6;
  sq = sum64(sq);
  sk = sum64(sk);
  if (lane == 0) red[wid] = sq, red2[wid] = sk;
  __syncthreads();
  sq = sk = 0.f;
#pragma unroll
  for (int i = 0; i < NTH / 64; ++i) sq += red[i], sk += red2[i];
  const float rq = p.qscale / sqrtf(sq + 1e-6f), rk = 1.f / sqrtf(sk + 1e-6f);
  const T* gates = proj + (int64_t)b * p.ldp + C + H * V;
  const float beta = sigmoidf_(ld(gates + h));
  const float gt = expf(-expf(p.a_log[h]) * softplusf_(ld(gates + H + h) + p.dt_bias[h]));
  f32x4_t k[NI], q[NI];
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    k[i] = ld4(&ks[i * 32 + l * 4]) * rk;
    q[i] = ld4(&qs[i * 32 + l * 4]) * rq;
  }
  float so = 0.f;
  for (int v = col; v < V; v += COLS) {
    float* sp = state + (int64_t)v * DP;
    if (v != col) {
#pragma unroll
      for (int i = 0; i < NI; ++i) S[i] = ld4(sp + i * 32 + l * 4);
    }
    float dot = 0.f;
#pragma unroll
    for (int i = 0; i < NI; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[i][e] = ps > 0 ? S[i][e] * gt : 0.f;   // a sequence's first token starts from zero
        dot += S[i][e] * k[i][e];
      }
    dot = sum8(dot);
    const float u = beta * (vs[v] - dot);
    float out = 0.f;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[i][e] += k[i][e] * u;
        out += S[i][e] * q[i][e];
      }
      st4(sp + i * 32 + l * 4, S[i]);
    }
    out = sum8(out);
    if (l == 0) {
      os[v] = out;
      so += out * out;
    }
  }
  so = sum64(so);   // (l == 0 lanes hold their columns' squares)
  if (lane == 0) red3[wid] = so;
  __syncthreads();
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NTH / 64; ++i) ss += red3[i];
  const float r = 1.f / sqrtf(ss / (float)V + p.eps);
  T* y = static_cast<T*>(p.y) + (int64_t)b * p.ldy + h * V;
  const T* gate = proj + (int64_t)b * p.ldp + C + h * V;
  for (int v = tid; v < V; v += NTH) st(y + v, os[v] * r * p.norm_w[v] * siluf_(ld(gate + v)));
}

#define NXD_BY_NI(CALL)                                                     \
  switch (p.DP / 32) {                                                      \
    case 1: CALL(1); break;                                                 \
    case 2: CALL(2); break;                                                 \
    case 3: CALL(3); break;                                                 \
    case 4: CALL(4); break;                                                 \
    case 5: CALL(5); break;                                                 \
    case 6: CALL(6); break;                                                 \
    case 7: CALL(7); break;                                                 \
    case 8: CALL(8); break;                                                 \
    default: return -1;                                                     \
  }

template <typename T>
static int run_prep(const DeltaParams& p, hipStream_t s) {
  const dim3 grid((unsigned)ceil_div(p.nch > 0 ? p.nch * 64 : p.T, PREP_TOKENS), (unsigned)p.B);
  const bool pairs = p.D % 2 == 0 && p.V % 2 == 0 && p.ldp % 2 == 0;
  if (pairs && p.DP <= 128) hipLaunchKernelGGL((delta_prep_kernel<T, 2, 1>), grid, dim3(256), 0, s, p);
  else if (pairs) hipLaunchKernelGGL((delta_prep_kernel<T, 2, 2>), grid, dim3(256), 0, s, p);
  else hipLaunchKernelGGL((delta_prep_kernel<T, 1, 4>), grid, dim3(256), 0, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 1;
}
template <typename T>
static int run_scan(const DeltaParams& p, hipStream_t s) {
  const dim3 grid((unsigned)ceil_div(p.V, 32), (unsigned)p.H, (unsigned)p.B);
#define NXD_CALL(N) hipLaunchKernelGGL((delta_scan_kernel<T, N>), grid, dim3(256), 0, s, p)
  NXD_BY_NI(NXD_CALL)
#undef NXD_CALL
  return hipGetLastError() == hipSuccess ? 0 : 1;
}
template <typename T>
static int run_out(const DeltaParams& p, hipStream_t s) {
  const int64_t n = (int64_t)p.B * p.T * p.H;
  const dim3 block(256);
#define NXD_OUT4(L) hipLaunchKernelGGL((delta_out4_kernel<T, L>), dim3((unsigned)ceil_div64(n, 256 / L)), block, 0, s, p)
  if (p.V % 4 || p.C % 4 || p.ldp % 4 || p.ldy % 4)
    hipLaunchKernelGGL((delta_out_kernel<T>), dim3((unsigned)ceil_div64(n, 4)), block, 0, s, p);
  else if (p.V <= 16) NXD_OUT4(4);
  else if (p.V <= 32) NXD_OUT4(8);
  else if (p.V <= 64) NXD_OUT4(16);
  else if (p.V <= 128) NXD_OUT4(32);
  else NXD_OUT4(64);
#undef NXD_OUT4
  return hipGetLastError() == hipSuccess ? 0 : 1;
}
template <typename T>
static int run_decode(const DeltaParams& p, hipStream_t s) {
  const dim3 grid((unsigned)p.H, (unsigned)p.B);
  if (p.V > 64) {
#define NXD_CALL(N) hipLaunchKernelGGL((delta_decode_kernel<T, N, 1024>), grid, dim3(1024), 0, s, p)
    NXD_BY_NI(NXD_CALL)
#undef NXD_CALL
  } else {
#define NXD_CALL(N) hipLaunchKernelGGL((delta_decode_kernel<T, N, 256>), grid, dim3(256), 0, s, p)
    NXD_BY_NI(NXD_CALL)
#undef NXD_CALL
  }
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

}  // namespace hybrid

int delta_prep_launch(bool f32, const DeltaParams& p, hipStream_t s) {
  return f32 ? hybrid::run_prep<float>(p, s) : hybrid::run_prep<uint16_t>(p, s);
}
int delta_scan_launch(bool f32, const DeltaParams& p, hipStream_t s) {
  return f32 ? hybrid::run_scan<float>(p, s) : hybrid::run_scan<uint16_t>(p, s);
}
int delta_out_launch(bool f32, const DeltaParams& p, hipStream_t s) {
  return f32 ? hybrid::run_out<float>(p, s) : hybrid::run_out<uint16_t>(p, s);
}
int delta_decode_launch(bool f32, const DeltaParams& p, hipStream_t s) {
  return f32 ? hybrid::run_decode<float>(p, s) : hybrid::run_decode<uint16_t>(p, s);
}

}  // namespace nxd
