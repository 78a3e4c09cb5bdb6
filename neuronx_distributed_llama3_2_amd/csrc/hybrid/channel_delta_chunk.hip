// Generalised delta rule over long runs of new tokens, a chunk of C at a time, on the fp32 matrix
// instructions.
//
// With L_t the running sum of the log decays of a chunk (per key channel) and b = -a u, define
//   U_t = u_t e^(L_(t-1)),  R_t = r_t e^(L_t),  B_t = b_t e^(-L_t),  K_t = k_t e^(-L_t)       (rows)
// The removals' read-outs z_t = u_t^T S_(t-1) of all tokens solve (A = strictly lower parts)
//   (I - A_ub) Z = U S_0 + A_uk V,     A_ub = U B^T, A_uk = U K^T
// which is linear in the state S_0 the chunk starts from: Z = W S_0 + Y.  With the lower parts (diagonal
// included) A_rb = R B^T, A_rk = R K^T and E = diag(e^(L_C)):
//   O   = Q S_0 + O',            Q = R + A_rb W,  O' = A_rb Y + A_rk V
//   S_1 = E S_0 + (E B^T) Z + (E K^T) V
//
//   prepare : Q, O', W, Y, E B^T, E K^T, V of every (sequence, chunk, head) in parallel
//   scan    : Z and the next state, the chunks of a head one after another for 16 columns of the state; a
//             wave has 16 rows of it, so W S_0 is summed over the waves (by waves of their own, while the others
//             multiply K^T V), and nothing else is exchanged
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
// N products, their steps interleaved (a step waits for the one before it in its own chain)
template <int N, typename A, typename B>
__device__ __forceinline__ void mma4_interleaved(A a, B b, f32x4_t (&c)[N]) {
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int n = 0; n < N; ++n) c[n] = __builtin_amdgcn_mfma_f32_16x16x4f32(a(n)[i], b(n)[i], c[n], 0, 0, 0);
}
// 2^x for a sum x kept in fp64
__device__ __forceinline__ float pow2(double x) {
  const double n = rint(x);
  return ldexpf(__builtin_amdgcn_exp2f((float)(x - n)), (int)n);
}

// a uniform base and a lane's offset in bytes: one address register a lane (the base is kept apart from the
// offset by hand, or the loop gets a 64-bit address a lane for every load)
template <typename V, typename P>
__device__ __forceinline__ V at(const P* base, uint32_t bytes) {
  typedef const __attribute__((address_space(1))) char* global_t;
  global_t g = (global_t)(const char*)base;
  asm("" : "+s"(g));
  return *(const __attribute__((address_space(1))) V*)(g + bytes);
}

constexpr int RANK_TILE = 64;

// 8 neighbouring elements of a row, all of them there and 16-byte aligned (`wide`) or not
template <typename T>
struct Raw8;
template <>
struct Raw8<uint16_t> {
  u32x4_t v;
  __device__ void load(const uint16_t* p) { v = *reinterpret_cast<const u32x4_t*>(p); }
  __device__ void zero() { v = u32x4_t{0u, 0u, 0u, 0u}; }
  __device__ void get(float (&f)[8]) const { unpack8(v, f); }
};
template <>
struct Raw8<float> {
  f32x4_t a, b;
  __device__ void load(const float* p) { a = ld4(p), b = ld4(p + 4); }
  __device__ void zero() { a = b = f32x4_t{0.f, 0.f, 0.f, 0.f}; }
  __device__ void get(float (&f)[8]) const {
#pragma unroll
    for (int i = 0; i < 4; ++i) f[i] = a[i], f[4 + i] = b[i];
  }
};

// LDS of the prepare kernel (floats): U, later the four products (with the rank tile before both); then R, B, K
template <int NB, int CB>
constexpr int first_region() {
  constexpr int C = CB * 16, u = C * (NB * 16 + 4), a = 4 * C * C, r = C * (RANK_TILE + 4);
  return u > a ? (u > r ? u : r) : (a > r ? a : r);
}

// NB = DP / 16 blocks of the head's channels, CB = C / 16 of the chunk's tokens.  One workgroup of 8 waves
// a cell.
template <typename T, int NB, int CB>
__global__ void __launch_bounds__(512, CB == 2 ? 4 : 2) cdelta_prepare_kernel(ChannelDeltaParams p) {
  constexpr int DP = NB * 16, C = CB * 16, KS = DP + 4;               // row stride of U, R, B, K
  constexpr int JW = (2 * NB + 7) / 8, HB = CB / 2, RS = RANK_TILE + 4;
  constexpr int LPT = 512 / C;                                        // lanes a token
  constexpr int PJ = CB * (CB + 1) / 2 * 4, PW = (PJ + 7) / 8;        // blocks of the products, of them a wave
  static_assert(C * DP / 8 <= 512, "a thread has 8 elements of a row");
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float *us = sm, *rs = us + first_region<NB, CB>(), *bs = rs + C * KS, *ks = bs + C * KS;   // [C][KS]
  float* am = us;   // A_ub, A_uk, A_rb, A_rk: [C][C] each, 16-byte pieces of a row swapped by its number
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
  // columns of V this wave solves for, and of U
  const int tv = w, tw = w >= NB ? w - NB : w + 8 - NB;
  const bool has_v = tv < NB && tv * 16 < D, has_w = tw < NB;

  // ---- r, k, removal are on their way first: 8 elements a thread
  const bool wide = D % 8 == 0 && p.ldp % 8 == 0 && reinterpret_cast<uintptr_t>(p.proj) % 16 == 0;
  const int rt = tid / (DP / 8), rc = tid % (DP / 8) * 8;
  Raw8<T> raw[3];
#pragma unroll
  for (int j = 0; j < 3; ++j) raw[j].zero();
  if (wide && rt < n && rc < D) {
#pragma unroll
    for (int j = 0; j < 3; ++j) raw[j].load(head + (int64_t)rt * p.ldp + (j == 0 ? 0 : (j == 1 ? HD : 4 * HD)) + rc);
  }

  // ---- log decays: W2 tanh(low), tokens x channels.  job = (channel block, half of the tokens)
  f32x4_t lw[JW][HB];
#pragma unroll
  for (int j = 0; j < JW; ++j)
#pragma unroll
    for (int i = 0; i < HB; ++i) lw[j][i] = zero;
  float* tl = us;   // [C][RS]
  for (int r0 = 0; r0 < N; r0 += RANK_TILE) {
    if (r0 > 0) __syncthreads();
    for (int i = tid; i < C * RANK_TILE; i += 512) {
      const int t = i / RANK_TILE, k = i % RANK_TILE;
      tl[t * RS + k] = t < n && r0 + k < N ? tanhf_(ld(head + (int64_t)t * p.ldp + 5 * HD - h * D + r0 + k)) : 0.f;
    }
    if (r0 == 0) {
      if (wide) {
        if (rt < C) {
#pragma unroll
          for (int j = 0; j < 3; ++j) {
            float f[8];
            raw[j].get(f);
            float* o = (j == 0 ? rs : (j == 1 ? ks : bs)) + rt * KS + rc;
            st4(o, f32x4_t{f[0], f[1], f[2], f[3]});
            st4(o + 4, f32x4_t{f[4], f[5], f[6], f[7]});
          }
        }
      } else {
        for (int i = tid; i < C * DP; i += 512) {
          const int t = i / DP, c = i % DP;
          const bool in = t < n && c < D;
          const T* x = head + (int64_t)t * p.ldp + c;
          rs[t * KS + c] = in ? ld(x) : 0.f;
          ks[t * KS + c] = in ? ld(x + HD) : 0.f;
          bs[t * KS + c] = in ? ld(x + 4 * HD) : 0.f;
        }
      }
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
        const int k = 16 * s + 4 * lq;
        f32x4_t f = zero;
        if (N % 4 == 0) {
          if (r0 + k < N) f = ld4(wr + k);
        } else {
#pragma unroll
          for (int i = 0; i < 4; ++i) f[i] = r0 + k + i < N ? ld(wr + k + i) : 0.f;
        }
#pragma unroll
        for (int i = 0; i < HB; ++i) lw[j][i] = mma4(ld4(tl + (16 * (half * HB + i) + lr) * RS + k), f, lw[j][i]);
      }
    }
  }
  {   // lengths of the keys
    const int t = tid / LPT, j = tid % LPT;
    float ss = 0.f;
    for (int d = 4 * j; d < DP; d += 4 * LPT) {
      const f32x4_t x = ld4(ks + t * KS + d);
      ss += x[0] * x[0] + x[1] * x[1] + x[2] * x[2] + x[3] * x[3];
    }
    ss = sum_lanes<LPT>(ss);
    if (j == 0) rn[t] = 1.f / sqrtf(ss + 1e-6f);
  }
  // the decays' running sums: of a half's tokens, then over both halves
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
  __syncthreads();   // (the rank tile's last readers are done as well)
  if (tid < DP) {
    ec[tid] = pow2(tot[0][tid] + tot[1][tid]);
    p.ce[cell * DP + tid] = ec[tid];
  }
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
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = 16 * (half * HB + i) + 4 * lq + e, o = t * KS + c;
        const float k = ks[o], u = k * rn[t], a = 1.f / (1.f + expf(-(bs[o] + ab)));
        us[o] = u * pow2(L);
        L += (double)lw[j][i][e];
        const float inv = pow2(-L);
        rs[o] *= pow2(L);
        bs[o] = -a * u * inv;
        ks[o] = k * inv;
      }
    }
  }
  __syncthreads();

  // ---- the lower blocks of the four products; this wave's columns of V, and of U before they go
  auto piece = [&](int m, int row, int ch16) { return am + (m * C + row) * C + 4 * (ch16 ^ (row & (C / 4 - 1))); };
  f32x4_t v[CB];
#pragma unroll
  for (int bk = 0; bk < CB; ++bk) {
    v[bk] = zero;
    if (has_v) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = 16 * bk + 4 * lq + i, col = tv * 16 + lr;
        if (t < n && col < D) v[bk][i] = ld(head + (int64_t)t * p.ldp + 2 * HD + col);
      }
    }
  }
  f32x4_t prod[PW], uw[CB];
#pragma unroll
  for (int j = 0; j < PW; ++j) {
    const int job = w + 8 * j;
    prod[j] = zero;
    if (job >= PJ) continue;
    int bi = 0, bj = job >> 2;
    while (bj > bi) bj -= ++bi;   // (0,0) (1,0) (1,1) (2,0) ...
    const float *ra = (job & 2) ? rs : us, *rb = (job & 1) ? ks : bs;
    f32x4_t x0 = zero, x1 = zero;
#pragma unroll
    for (int kb = 0; kb < NB; kb += 2) {   // NB is even
      const int ro = (16 * bi + lr) * KS + 16 * kb + 4 * lq, co = (16 * bj + lr) * KS + 16 * kb + 4 * lq;
      x0 = mma4(ld4(ra + ro), ld4(rb + co), x0);
      x1 = mma4(ld4(ra + ro + 16), ld4(rb + co + 16), x1);
    }
    prod[j] = x0 + x1;
  }
#pragma unroll
  for (int bi = 0; bi < CB; ++bi)
#pragma unroll
    for (int i = 0; i < 4; ++i) uw[bi][i] = has_w ? us[(16 * bi + 4 * lq + i) * KS + tw * 16 + lr] : 0.f;
  __syncthreads();
#pragma unroll
  for (int j = 0; j < PW; ++j) {
    const int job = w + 8 * j, m = job & 3;
    if (job >= PJ) continue;
    int bi = 0, bj = job >> 2;
    while (bj > bi) bj -= ++bi;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int row = 16 * bi + 4 * lq + i, col = 16 * bj + lr;
      piece(m, row, col >> 2)[col & 3] = col < row || (m >= 2 && col == row) ? prod[j][i] : 0.f;
    }
  }
  __syncthreads();

  // ---- the diagonal blocks of I - A_ub, inverted in place by substitution: column lr
  if (w < CB) {
    float x[16];
    auto el = [&](int i, int j) { return piece(0, 16 * w + i, 4 * w + (j >> 2)) + (j & 3); };
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float s = i == lr ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < i; ++j) s += *el(i, j) * x[j];
      x[i] = s;
    }
    __builtin_amdgcn_wave_barrier();
    if (lq == 0) {
#pragma unroll
      for (int i = 0; i < 16; ++i) *el(i, lr) = x[i];
    }
  }
  // ---- E B^T and E K^T, A operands of the scan
  for (int job = w; job < NB * CB; job += 8) {
    const int cb = job / CB, bk = job % CB;
    const float e = ec[16 * cb + lr];
    f32x4_t fb, fk;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int o = (16 * bk + 4 * lq + i) * KS + 16 * cb + lr;
      fb[i] = bs[o] * e;
      fk[i] = ks[o] * e;
    }
    st4(p.cb + ((cell * NB + cb) * CB + bk) * 256 + lane * 4, fb);
    st4(p.ck + ((cell * NB + cb) * CB + bk) * 256 + lane * 4, fk);
  }
  __syncthreads();

  // ---- 16 columns of Y (from V) and of W (from U), and the outputs' parts
  auto frag = [&](int m, int bi, int bk) { return ld4(piece(m, 16 * bi + lr, 4 * bk + lq)); };
  if (has_v) {
    f32x4_t y[CB];
#pragma unroll
    for (int bi = 0; bi < CB; ++bi) {
      st4(p.cv + ((cell * NB + tv) * CB + bi) * 256 + lane * 4, v[bi]);
      f32x4_t r = zero;
#pragma unroll
      for (int bk = 0; bk <= bi; ++bk) r = mma4(frag(1, bi, bk), v[bk], r);
#pragma unroll
      for (int bk = 0; bk < bi; ++bk) r = mma4(frag(0, bi, bk), y[bk], r);
      y[bi] = mma4(frag(0, bi, bi), r, zero);
      st4(p.cy + ((cell * NB + tv) * CB + bi) * 256 + lane * 4, y[bi]);
    }
#pragma unroll
    for (int bi = 0; bi < CB; ++bi) {
      f32x4_t o = zero, o2 = zero;
#pragma unroll
      for (int bk = 0; bk <= bi; ++bk) {
        o = mma4(frag(2, bi, bk), y[bk], o);
        o2 = mma4(frag(3, bi, bk), v[bk], o2);
      }
      st4(p.co + ((cell * NB + tv) * CB + bi) * 256 + lane * 4, o + o2);
    }
  }
  if (has_w) {
    f32x4_t y[CB];
#pragma unroll
    for (int bi = 0; bi < CB; ++bi) {
      f32x4_t r = uw[bi];
#pragma unroll
      for (int bk = 0; bk < bi; ++bk) r = mma4(frag(0, bi, bk), y[bk], r);
      y[bi] = mma4(frag(0, bi, bi), r, zero);
      // W as an A operand: its transpose is what these registers are
      float* o = p.cw + ((cell * NB + tw) * CB + bi) * 256 + (lr >> 2) * 64 + (lr & 3);
#pragma unroll
      for (int i = 0; i < 4; ++i) o[(4 * lq + i) * 4] = y[bi][i];
    }
#pragma unroll
    for (int bi = 0; bi < CB; ++bi) {   // (a transposed product: an A operand of what reads it)
      f32x4_t q = ld4(rs + (16 * bi + lr) * KS + 16 * tw + 4 * lq);
#pragma unroll
      for (int bk = 0; bk <= bi; ++bk) q = mma4(y[bk], frag(2, bi, bk), q);
      st4(p.cq + ((cell * CB + bi) * NB + tw) * 256 + lane * 4, q);
    }
  }
}

// 16 columns of one head's state: a wave for 16 rows of it, and a wave for 16 tokens that sums the waves' parts
// of W S_0.  A chunk's operands are fetched AHEAD chunks before.
template <int NB, int CB>
__global__ void __launch_bounds__((NB + CB) * 64) cdelta_scan_kernel(ChannelDeltaParams p) {
  constexpr int DP = NB * 16, C = CB * 16, AHEAD = CB == 2 ? 3 : 2;
  __shared__ __attribute__((aligned(16))) f32x4_t part[NB][CB][64], zs[CB][64];
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lq = lane >> 4;
  const int bh = blockIdx.x % (p.B * p.H), vt = blockIdx.x / (p.B * p.H);   // a head's columns on one XCD
  const int b = bh / p.H, h = bh % p.H, H = p.H, D = p.D, v = vt * 16 + lr;
  const int len = p.lens ? min(p.lens[b], p.T) : p.T;
  if (len <= 0) return;
  const int nch = (len + C - 1) / C;
  const int64_t NC = (int64_t)NB * CB * 256;   // floats of a cell's operand
  const uint32_t l16 = lane * 16;
  auto cell_of = [&](int c) { return ((int64_t)b * p.nch + min(c, nch - 1)) * H + h; };   // (past the end the last is read again)
  if (w >= NB) {
    const int blk = w - NB;
    const float* y = p.cy + (vt * CB + blk) * 256;
    f32x4_t set[AHEAD];
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) set[i] = at<f32x4_t>(y + cell_of(i) * NC, l16);
    auto chunk = [&](int c, f32x4_t& o) {
      lds_barrier();
      f32x4_t z = part[0][blk][lane];
#pragma unroll
      for (int j = 1; j < NB; ++j) z += part[j][blk][lane];
      zs[blk][lane] = z + o;
      __builtin_amdgcn_sched_barrier(0);   // a load ahead of the old value's last use would need a register of its own,
      o = at<f32x4_t>(y + cell_of(c + AHEAD) * NC, l16);   // and a copy that waits for it
      lds_barrier();
    };
    int c = 0;
    for (; c + AHEAD <= nch; c += AHEAD) {
#pragma unroll
      for (int i = 0; i < AHEAD; ++i) chunk(c + i, set[i]);
    }
#pragma unroll
    for (int i = 0; i < AHEAD; ++i)
      if (c + i < nch) chunk(c + i, set[i]);
    return;
  }
  const int slot = slot_of(p.slots, b, p.nslots);
  const int64_t p0 = pos_of(p.pos, p.pos_stride, b);
  float* state = p.state + (((int64_t)slot * H + h) * D + min(v, D - 1)) * DP + w * 16 + 4 * lq;
  const f32x4_t zero = {0.f, 0.f, 0.f, 0.f};
  f32x4_t S = zero;
  if (p0 > 0 && v < D) S = ld4(state);
  struct Ops {
    f32x4_t w[CB], k[CB], v[CB], b[CB], e;
  };
  Ops set[AHEAD];
  auto fetch_first = [&](int c, Ops& o) {
    const int64_t cell = cell_of(c), first = cell * NC + w * CB * 256;   // (uniform)
#pragma unroll
    for (int i = 0; i < CB; ++i) {
      o.w[i] = at<f32x4_t>(p.cw + first + i * 256, l16);
      o.k[i] = at<f32x4_t>(p.ck + first + i * 256, l16);
      o.v[i] = at<f32x4_t>(p.cv + cell * NC + (vt * CB + i) * 256, l16);
    }
    o.e = at<f32x4_t>(p.ce + cell * DP + w * 16, lq * 16);
  };
  auto fetch_last = [&](int c, Ops& o) {
    const float* src = p.cb + cell_of(c) * NC + w * CB * 256;
#pragma unroll
    for (int i = 0; i < CB; ++i) o.b[i] = at<f32x4_t>(src + i * 256, l16);
  };
#pragma unroll
  for (int i = 0; i < AHEAD; ++i) {
    fetch_first(i, set[i]);
    fetch_last(i, set[i]);
  }
  auto chunk = [&](int c, Ops& o) {
    f32x4_t z[CB];
#pragma unroll
    for (int i = 0; i < CB; ++i) z[i] = zero;
    mma4_interleaved<CB>([&](int i) { return o.w[i]; }, [&](int) { return S; }, z);
#pragma unroll
    for (int i = 0; i < CB; ++i) part[w][i][lane] = z[i];
    *reinterpret_cast<f32x4_t*>(reinterpret_cast<char*>(p.cs + ((cell_of(c) * NB + vt) * NB + w) * 256) + l16) = S;
    lds_barrier();
    z[0] = S * o.e;   // while the parts are summed: E S_0 + (E K^T) V
#pragma unroll
    for (int i = 1; i < CB; ++i) z[i] = zero;
    mma4_interleaved<CB>([&](int i) { return o.k[i]; }, [&](int i) { return o.v[i]; }, z);
    __builtin_amdgcn_sched_barrier(0);   // (as above)
    fetch_first(c + AHEAD, o);
    lds_barrier();
    f32x4_t x[CB];
#pragma unroll
    for (int i = 0; i < CB; ++i) x[i] = zs[i][lane];
    mma4_interleaved<CB>([&](int i) { return o.b[i]; }, [&](int i) { return x[i]; }, z);
    __builtin_amdgcn_sched_barrier(0);
    fetch_last(c + AHEAD, o);
    S = z[0];
#pragma unroll
    for (int i = 1; i < CB; ++i) S += z[i];
  };
  int c = 0;
  for (; c + AHEAD <= nch; c += AHEAD) {
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) chunk(c + i, set[i]);
  }
#pragma unroll
  for (int i = 0; i < AHEAD; ++i)
    if (c + i < nch) chunk(c + i, set[i]);
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
  constexpr size_t lds = (size_t)(first_region<NB, CB>() + 3 * C * (NB * 16 + 4)) * 4;
  static_assert(lds <= 152 * 1024, "LDS of a compute unit");
  static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(&cdelta_prepare_kernel<T, NB, CB>),
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
  if (attr != hipSuccess) return 2;
  const dim3 grid((unsigned)p.H, (unsigned)p.nch, (unsigned)p.B);
  hipLaunchKernelGGL((cdelta_prepare_kernel<T, NB, CB>), grid, dim3(512), lds, s, p);
  if (hipGetLastError() != hipSuccess) return 1;
  hipLaunchKernelGGL((cdelta_scan_kernel<NB, CB>), dim3((unsigned)(ceil_div(p.D, 16) * p.B * p.H)), dim3((NB + CB) * 64), 0, s, p);
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
