// Generalised delta rule over long runs of new tokens, a chunk of C at a time, on the fp32 matrix
// instructions.
//
// With L_t the running sum of the log decays of a chunk (per key channel) and b = -a u, define
//   U_t = u_t e^(L_(t-1)),  R_t = r_t e^(L_t),  B_t = b_t e^(-L_t),  K_t = k_t e^(-L_t)       (rows)
// The removals' read-outs z_t = u_t^T S_(t-1) of all tokens solve (A = strictly lower parts)
//   (I - A_ub) Z = U S_0 + A_uk V,     A_ub = U B^T, A_uk = U K^T
// which is linear in the state S_0 the chunk starts from: Z = W S_0 + Y.  With the lower parts (diagonal
// included) A_rb = R B^T, A_rk = R K^T and E = diag(e^(L_C)) everything else is linear in S_0 as well:
//   O   = Q S_0 + O',   Q = R + A_rb W,        O' = A_rb Y + A_rk V
//   S_1 = T S_0 + M,    T = E (I + B^T W),     M  = E (B^T Y + K^T V)
//
//   prepare : Q, O', T, M of every (sequence, chunk, head) in parallel
//   scan    : S <- T S + M, the chunks of a head one after another for 16 columns of the state
//   output  : O = Q S_0 + O', the head norm and the gate
//
// A log decay lies in (-e^(-1/2), 0), so e^(-L) stays below e^39 in a chunk of 64 and every product of a
// factor with its counterpart is formed from two fp32 numbers of full precision: the sums are fp64, the
// exponentials are split into 2^n and 2^f.
//
// Fragments.  Of a 16 x 16 block, lane l holds the four elements [4 (l / 16) + i][l % 16], i < 4: the
// result layout of v_mfma_f32_16x16x4_f32.  Taken over k in the order 4 (l / 16) + i, the same registers
// are a B operand, and the A operand of the transposed block, so results feed the next product without
// moving.  What the later kernels read is stored block by block in the order of its lanes (1 KiB a block).
#include "channel_delta.h"

namespace nxd {
namespace hybrid {

__device__ __forceinline__ f32x4_t mma4(const f32x4_t& a, const f32x4_t& b, f32x4_t c) {
#pragma unroll
  for (int i = 0; i < 4; ++i) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[i], c, 0, 0, 0);
  return c;
}
// 2^x for a sum x kept in fp64
__device__ __forceinline__ float pow2(double x) {
  const double n = rint(x);
  return ldexpf(__builtin_amdgcn_exp2f((float)(x - n)), (int)n);
}

constexpr int RANK_TILE = 64;

// NB = DP / 16 blocks of the head's channels, CB = C / 16 of the chunk's tokens.  One workgroup of 8 waves
// a cell.
template <typename T, int NB, int CB>
__global__ void __launch_bounds__(512) cdelta_prepare_kernel(ChannelDeltaParams p) {
  constexpr int DP = NB * 16, C = CB * 16, KS = DP + 4, AS = C + 4;   // LDS row strides (floats)
  constexpr int JW = (2 * NB + 7) / 8, HB = CB / 2, RS = RANK_TILE + 4;
  constexpr int LPT = 512 / C;                                        // lanes a token
  static_assert(C * RS <= 4 * C * AS, "the rank tile fits where the products go");
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float *us = sm, *rs = us + C * KS, *bs = rs + C * KS, *ks = bs + C * KS;   // [C][KS]
  float* am = ks + C * KS;                                                   // A_ub, A_uk, A_rb, A_rk: [C][AS] each
  __shared__ float rn[C], ec[DP];
  __shared__ double tot[2][DP];
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lq = lane >> 4;
  const int h = blockIdx.x, ch = blockIdx.y, b = blockIdx.z, H = p.H, D = p.D, N = p.N, HD = H * D;
  const int len = p.lens ? min(p.lens[b], p.T) : p.T;
  const int n = min(C, len - ch * C);
  if (n <= 0) return;
  const int64_t m0 = (int64_t)b * p.T + ch * C;
  const int64_t cell = ((int64_t)b * p.nch + ch) * H + h;
  const T* head = static_cast<const T*>(p.proj) + m0 * p.ldp + h * D;
  const f32x4_t zero = {0.f, 0.f, 0.f, 0.f};

  {   // ---- lengths of the keys
    const int t = tid / LPT, j = tid % LPT;
    float ss = 0.f;
    if (t < n) {
      const T* k = head + (int64_t)t * p.ldp + HD;
      if (D % 4 == 0 && p.ldp % 4 == 0 && reinterpret_cast<uintptr_t>(p.proj) % 16 == 0) {
        for (int d = 4 * j; d < D; d += 4 * LPT) {
          const f32x4_t v = ld4(k + d);
          ss += v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
        }
      } else {
        for (int d = j; d < D; d += LPT) {
          const float v = ld(k + d);
          ss += v * v;
        }
      }
    }
    ss = sum_lanes<LPT>(ss);
    if (j == 0) rn[t] = 1.f / sqrtf(ss + 1e-6f);
  }

  // ---- log decays: W2 tanh(low), tokens x channels.  job = (channel block, half of the tokens)
  f32x4_t lw[JW][HB];
#pragma unroll
  for (int j = 0; j < JW; ++j)
#pragma unroll
    for (int i = 0; i < HB; ++i) lw[j][i] = zero;
  float* tl = am;   // [C][RS]
  for (int r0 = 0; r0 < N; r0 += RANK_TILE) {
    __syncthreads();
    for (int i = tid; i < C * RANK_TILE; i += 512) {
      const int t = i / RANK_TILE, k = i % RANK_TILE;
      tl[t * RS + k] = t < n && r0 + k < N ? tanhf_(ld(head + (int64_t)t * p.ldp + 5 * HD - h * D + r0 + k)) : 0.f;
    }
    __syncthreads();
    const int steps = (min(N - r0, RANK_TILE) + 15) / 16;
#pragma unroll
    for (int j = 0; j < JW; ++j) {
      const int job = w + 8 * j;
      if (job >= 2 * NB) continue;
      const int c = (job % NB) * 16 + lr, half = job / NB;
      const T* wr = static_cast<const T*>(p.w2) + (int64_t)(h * D + min(c, D - 1)) * N + r0;
      for (int s = 0; s < steps; ++s) {
        f32x4_t f;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int k = 16 * s + 4 * lq + i;
          f[i] = r0 + k < N ? ld(wr + k) : 0.f;
        }
#pragma unroll
        for (int i = 0; i < HB; ++i) lw[j][i] = mma4(ld4(tl + (16 * (half * HB + i) + lr) * RS + 16 * s + 4 * lq), f, lw[j][i]);
      }
    }
  }
  // their running sums: of a half's tokens, then over both halves
  double base[JW][HB];   // sum before the lane's four tokens of a block
#pragma unroll
  for (int j = 0; j < JW; ++j) {
    const int job = w + 8 * j;
    if (job >= 2 * NB) continue;
    const int c = (job % NB) * 16 + lr, half = job / NB;
    const float w0 = c < D ? p.w0[h * D + c] : 0.f;
    double run = 0.0;
#pragma unroll
    for (int i = 0; i < HB; ++i) {
      double sum = 0.0;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = 16 * (half * HB + i) + 4 * lq + e;
        lw[j][i][e] = t < n && c < D ? decay_log2(lw[j][i][e] + w0) : 0.f;
        sum += (double)lw[j][i][e];
      }
      double s = sum, q = __shfl_up(s, 16, 64);
      if (lq >= 1) s += q;
      q = __shfl_up(s, 32, 64);
      if (lq >= 2) s += q;
      base[j][i] = run + s - sum;
      run += __shfl(s, 48 + lr, 64);
    }
    if (lq == 0) tot[half][c] = run;
  }
  __syncthreads();
  if (tid < DP) ec[tid] = pow2(tot[0][tid] + tot[1][tid]);
#pragma unroll
  for (int j = 0; j < JW; ++j) {
    const int job = w + 8 * j;
    if (job >= 2 * NB) continue;
    const int c = (job % NB) * 16 + lr, half = job / NB;
    const float ab = c < D ? p.a_bias[h * D + c] : 0.f;
    const double before = half ? tot[0][c] : 0.0;
#pragma unroll
    for (int i = 0; i < HB; ++i) {
      double L = before + base[j][i];
      float kk[4], aa[4], rr[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = 16 * (half * HB + i) + 4 * lq + e;
        const bool in = t < n && c < D;
        const T* x = head + (int64_t)min(t, n - 1) * p.ldp + min(c, D - 1);
        kk[e] = in ? ld(x + HD) : 0.f;
        aa[e] = ld(x + 4 * HD);
        rr[e] = in ? ld(x) : 0.f;
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = 16 * (half * HB + i) + 4 * lq + e, o = t * KS + c;
        const float u = kk[e] * rn[t], a = 1.f / (1.f + expf(-(aa[e] + ab)));
        us[o] = u * pow2(L);
        L += (double)lw[j][i][e];
        const float inv = pow2(-L);
        rs[o] = rr[e] * pow2(L);
        bs[o] = -a * u * inv;
        ks[o] = kk[e] * inv;
      }
    }
  }
  __syncthreads();

  // ---- the lower blocks of the four products
  for (int job = w; job < CB * (CB + 1) / 2; job += 8) {
    int bi = 0, bj = job;
    while (bj > bi) bj -= ++bi;   // (0,0) (1,0) (1,1) (2,0) ...
    f32x4_t ub = zero, uk = zero, rb = zero, rk = zero;
#pragma unroll
    for (int kb = 0; kb < NB; ++kb) {
      const int ro = (16 * bi + lr) * KS + 16 * kb + 4 * lq, co = (16 * bj + lr) * KS + 16 * kb + 4 * lq;
      const f32x4_t fu = ld4(us + ro), fr = ld4(rs + ro), fb = ld4(bs + co), fk = ld4(ks + co);
      ub = mma4(fu, fb, ub);
      uk = mma4(fu, fk, uk);
      rb = mma4(fr, fb, rb);
      rk = mma4(fr, fk, rk);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int row = 16 * bi + 4 * lq + i, col = 16 * bj + lr, o = row * AS + col;
      am[o] = col < row ? ub[i] : 0.f;
      am[C * AS + o] = col < row ? uk[i] : 0.f;
      am[2 * C * AS + o] = col <= row ? rb[i] : 0.f;
      am[3 * C * AS + o] = col <= row ? rk[i] : 0.f;
    }
  }
  __syncthreads();

  // ---- the diagonal blocks of I - A_ub, inverted in place by substitution: column lr
  if (w < CB) {
    float x[16];
    float* a = am + (16 * w) * AS + 16 * w;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float s = i == lr ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < i; ++j) s += a[i * AS + j] * x[j];
      x[i] = s;
    }
    __builtin_amdgcn_wave_barrier();
    if (lq == 0) {
#pragma unroll
      for (int i = 0; i < 16; ++i) a[i * AS + lr] = x[i];
    }
  }
  __syncthreads();

  // ---- 16 columns of Y (from V) or W (from U) at a time, and what follows from them
  auto frag = [&](int m, int bi, int bk) { return ld4(am + m * (C * AS) + (16 * bi + lr) * AS + 16 * bk + 4 * lq); };
  for (int tile = w; tile < 2 * NB; tile += 8) {
    const bool isv = tile < NB;
    const int col = (isv ? tile : tile - NB) * 16 + lr, cb0 = isv ? tile : tile - NB;
    if (isv && cb0 * 16 >= D) continue;
    f32x4_t y[CB], v[CB];
    if (isv) {
#pragma unroll
      for (int bk = 0; bk < CB; ++bk)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int t = 16 * bk + 4 * lq + i;
          v[bk][i] = t < n && col < D ? ld(head + (int64_t)t * p.ldp + 2 * HD + col) : 0.f;
        }
    }
#pragma unroll
    for (int bi = 0; bi < CB; ++bi) {
      f32x4_t r = zero;
      if (isv) {
#pragma unroll
        for (int bk = 0; bk <= bi; ++bk) r = mma4(frag(1, bi, bk), v[bk], r);
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i) r[i] = us[(16 * bi + 4 * lq + i) * KS + col];
      }
#pragma unroll
      for (int bk = 0; bk < bi; ++bk) r = mma4(frag(0, bi, bk), y[bk], r);
      y[bi] = mma4(frag(0, bi, bi), r, zero);
    }
    if (isv) {
#pragma unroll
      for (int bi = 0; bi < CB; ++bi) {
        f32x4_t o = zero, o2 = zero;
#pragma unroll
        for (int bk = 0; bk <= bi; ++bk) {
          o = mma4(frag(2, bi, bk), y[bk], o);
          o2 = mma4(frag(3, bi, bk), v[bk], o2);
        }
        st4(p.co + ((cell * NB + cb0) * CB + bi) * 256 + lane * 4, o + o2);
      }
#pragma unroll
      for (int cb = 0; cb < NB; ++cb) {
        f32x4_t m = zero, m2 = zero;
#pragma unroll
        for (int bk = 0; bk < CB; ++bk) {
          f32x4_t fb, fk;
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int o = (16 * bk + 4 * lq + i) * KS + 16 * cb + lr;
            fb[i] = bs[o];
            fk[i] = ks[o];
          }
          m = mma4(fb, y[bk], m);
          m2 = mma4(fk, v[bk], m2);
        }
        m += m2;
#pragma unroll
        for (int i = 0; i < 4; ++i) m[i] *= ec[16 * cb + 4 * lq + i];
        st4(p.cm + ((cell * NB + cb0) * NB + cb) * 256 + lane * 4, m);
      }
    } else {   // (transposed products: A operands of what reads them)
#pragma unroll
      for (int bi = 0; bi < CB; ++bi) {
        f32x4_t q = ld4(rs + (16 * bi + lr) * KS + 16 * cb0 + 4 * lq);
#pragma unroll
        for (int bk = 0; bk <= bi; ++bk) q = mma4(y[bk], frag(2, bi, bk), q);
        st4(p.cq + ((cell * CB + bi) * NB + cb0) * 256 + lane * 4, q);
      }
#pragma unroll
      for (int cb = 0; cb < NB; ++cb) {
        f32x4_t t = zero;
#pragma unroll
        for (int bk = 0; bk < CB; ++bk) {
          f32x4_t fb;
#pragma unroll
          for (int i = 0; i < 4; ++i) fb[i] = bs[(16 * bk + 4 * lq + i) * KS + 16 * cb + lr];
          t = mma4(y[bk], fb, t);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) t[i] = (t[i] + (16 * cb + lr == 16 * cb0 + 4 * lq + i ? 1.f : 0.f)) * ec[16 * cb + lr];
        st4(p.ct + ((cell * NB + cb) * NB + cb0) * 256 + lane * 4, t);
      }
    }
  }
}

// 16 columns of one head's state, a wave for 16 rows.  T and M are fetched four chunks ahead.
template <int NB, int CB>
__global__ void __launch_bounds__(NB * 64) cdelta_scan_kernel(ChannelDeltaParams p) {
  constexpr int DP = NB * 16, C = CB * 16, AHEAD = 4;
  __shared__ __attribute__((aligned(16))) f32x4_t ss[2][NB][64];
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lq = lane >> 4;
  const int bh = blockIdx.x % (p.B * p.H), vt = blockIdx.x / (p.B * p.H);   // a head's columns on one XCD
  const int b = bh / p.H, h = bh % p.H, H = p.H, D = p.D, v = vt * 16 + lr;
  const int len = p.lens ? min(p.lens[b], p.T) : p.T;
  if (len <= 0) return;
  const int slot = slot_of(p.slots, b, p.nslots);
  const int64_t p0 = pos_of(p.pos, p.pos_stride, b);
  float* state = p.state + (((int64_t)slot * H + h) * D + min(v, D - 1)) * DP + w * 16 + 4 * lq;
  f32x4_t S = {0.f, 0.f, 0.f, 0.f};
  if (p0 > 0 && v < D) S = ld4(state);
  const int nch = (len + C - 1) / C;
  struct Ops {
    f32x4_t t[NB], m;
  };
  Ops set[AHEAD];
  auto fetch = [&](int c, Ops& o) {   // (past the last chunk the last one is read again)
    const int64_t cell = ((int64_t)b * p.nch + min(c, nch - 1)) * H + h;
    const float* t = p.ct + (cell * NB + w) * (NB * 256) + lane * 4;
#pragma unroll
    for (int kb = 0; kb < NB; ++kb) o.t[kb] = ld4(t + kb * 256);
    o.m = ld4(p.cm + ((cell * NB + vt) * NB + w) * 256 + lane * 4);
  };
#pragma unroll
  for (int i = 0; i < AHEAD; ++i) fetch(i, set[i]);
  auto chunk = [&](int c, Ops& o, int flip) {
    const int64_t cell = ((int64_t)b * p.nch + c) * H + h;
    ss[flip][w][lane] = S;
    st4(p.cs + ((cell * NB + vt) * NB + w) * 256 + lane * 4, S);
    lds_barrier();
    f32x4_t s[NB], a0 = o.m, a1 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kb = 0; kb < NB; ++kb) s[kb] = ss[flip][kb][lane];
#pragma unroll
    for (int kb = 0; kb < NB; kb += 2) {   // NB is even
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.t[kb][i], s[kb][i], a0, 0, 0, 0);
        a1 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.t[kb + 1][i], s[kb + 1][i], a1, 0, 0, 0);
      }
    }
    S = a0 + a1;
    fetch(c + AHEAD, o);
  };
  int c = 0;
  for (; c + AHEAD <= nch; c += AHEAD) {
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) chunk(c + i, set[i], i & 1);
  }
#pragma unroll
  for (int i = 0; i < AHEAD; ++i)
    if (c + i < nch) chunk(c + i, set[i], i & 1);
  if (v < D) st4(state, S);
}

// A cell's outputs, a wave for 16 tokens.
template <typename T, int NB, int CB>
__global__ void __launch_bounds__(CB * 64) cdelta_output_kernel(ChannelDeltaParams p) {
  constexpr int C = CB * 16;
  const int tid = threadIdx.x, lane = tid & 63, bi = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lq = lane >> 4;
  const int h = blockIdx.x, ch = blockIdx.y, b = blockIdx.z, H = p.H, D = p.D;
  const int len = p.lens ? min(p.lens[b], p.T) : p.T;
  const int t0 = ch * C + 16 * bi + 4 * lq;   // the lane's four tokens
  T* y = static_cast<T*>(p.y) + ((int64_t)b * p.T + t0) * p.ldy + h * D + lr;
  const int nv = (D + 15) / 16;
  f32x4_t o[NB];
  float f[4] = {0.f, 0.f, 0.f, 0.f};
  if (ch * C < len) {   // (uniform)
    const int64_t cell = ((int64_t)b * p.nch + ch) * H + h;
    f32x4_t q[NB], ss = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kb = 0; kb < NB; ++kb) q[kb] = ld4(p.cq + ((cell * CB + bi) * NB + kb) * 256 + lane * 4);
#pragma unroll
    for (int vt = 0; vt < NB; ++vt) {
      o[vt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      if (vt >= nv) continue;
      const float* s = p.cs + (cell * NB + vt) * (NB * 256) + lane * 4;
      f32x4_t a = ld4(p.co + ((cell * NB + vt) * CB + bi) * 256 + lane * 4), a2 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kb = 0; kb < NB; kb += 2) {
        a = mma4(q[kb], ld4(s + kb * 256), a);
        a2 = mma4(q[kb + 1], ld4(s + (kb + 1) * 256), a2);
      }
      o[vt] = a + a2;
      ss += o[vt] * o[vt];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) f[i] = p.out_scale / sqrtf(sum16(ss[i]) / (float)D + p.eps);
  }
  const T* g = static_cast<const T*>(p.proj) + ((int64_t)b * p.T + t0) * p.ldp + 3 * H * D + h * D + lr;
#pragma unroll
  for (int vt = 0; vt < NB; ++vt) {
    if (vt * 16 + lr >= D) continue;
    const float nw = p.norm_w[h * D + vt * 16 + lr];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if (t0 + i >= p.T) continue;
      float x = 0.f;   // padding: a defined value for the projection
      if (t0 + i < len) x = o[vt][i] * f[i] * nw * sigmoidf_(ld(g + i * p.ldp + vt * 16));
      st(y + i * p.ldy + vt * 16, x);
    }
  }
}

template <typename T, int NB, int CB>
static int run_chunk(const ChannelDeltaParams& p, hipStream_t s) {
  constexpr int C = CB * 16;
  constexpr size_t lds = (size_t)4 * C * (NB * 16 + 4 + C + 4) * 4;
  static_assert(lds <= 152 * 1024, "LDS of a compute unit");
  static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(&cdelta_prepare_kernel<T, NB, CB>),
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
  if (attr != hipSuccess) return 2;
  const dim3 grid((unsigned)p.H, (unsigned)p.nch, (unsigned)p.B);
  hipLaunchKernelGGL((cdelta_prepare_kernel<T, NB, CB>), grid, dim3(512), lds, s, p);
  if (hipGetLastError() != hipSuccess) return 1;
  hipLaunchKernelGGL((cdelta_scan_kernel<NB, CB>), dim3((unsigned)(ceil_div(p.D, 16) * p.B * p.H)), dim3(NB * 64), 0, s, p);
  if (hipGetLastError() != hipSuccess) return 1;
  hipLaunchKernelGGL((cdelta_output_kernel<T, NB, CB>), grid, dim3(CB * 64), 0, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

template <typename T>
static int dispatch_cdelta(const ChannelDeltaParams& p, hipStream_t s) {
  switch (p.DP / 32) {
    case 1: return run_chunk<T, 2, 4>(p, s);
    case 2: return run_chunk<T, 4, 4>(p, s);
    case 3: return run_chunk<T, 6, 2>(p, s);
    case 4: return run_chunk<T, 8, 2>(p, s);
  }
  return -1;
}

}  // namespace hybrid

// tokens of a chunk for this head size (0: no chunked form)
int channel_delta_chunk(int DP) { return DP <= 64 ? 64 : (DP <= 128 ? 32 : 0); }
int channel_delta_chunk_launch(bool f32, const ChannelDeltaParams& p, hipStream_t s) {
  return f32 ? hybrid::dispatch_cdelta<float>(p, s) : hybrid::dispatch_cdelta<uint16_t>(p, s);
}

}  // namespace nxd
