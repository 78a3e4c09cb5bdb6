// Gated delta rule over long runs of new tokens, 64 at a time, on the fp32 matrix instructions.
//
// Within a chunk, with G_t the running sum of the log decays, the writes u_t of all its tokens solve
//   (I + A) U = diag(beta) (V - diag(e^G) K S_0),   A[t][s] = beta_t e^(G_t - G_s) k_t . k_s   (s < t)
// which is linear in the state S_0 the chunk starts from:  U = Y - W S_0.  Then
//   O   = diag(e^G) Q S_0 + P U,      P[t][s] = e^(G_t - G_s) q_t . k_s   (s <= t)
//   S_1 = e^(G_C) S_0 + K^T diag(e^(G_C - G)) U
//
//   delta_chunk_prepare : Y, W, P of every chunk and head in parallel: products of the chunk's keys and
//                         queries, the four 16 x 16 diagonal blocks of I + A inverted by substitution,
//                         the rest by block substitution with the right-hand sides in registers;
//   delta_chunk_scan    : the chunks of one head one after another for 16 columns of the state.
//
// Everything is fp32 (v_mfma_f32_16x16x4_f32); the sums of log decays are formed in fp64, because the
// differences of large sums are what is exponentiated.
//
// Fragments.  Of a 16 x 16 block, lane l holds the four elements [4 (l / 16) + i][l % 16], i < 4: the
// instruction's result layout.  Taken over k in the order 4 (l / 16) + i, the same registers are a B
// operand, so results feed the next product without moving; an A operand's lane holds four consecutive
// elements of row l % 16.  Everything the scan reads is stored block by block in the order of its lanes
// (1 KiB a block, element ((l / 16) 16 + l % 16) 4 + i): a block is one contiguous load.
#include "delta_rule.h"

namespace nxd {
namespace hybrid {

constexpr int CH = 64;   // tokens of a chunk

__device__ __forceinline__ f32x4_t mma4(const f32x4_t& a, const f32x4_t& b, f32x4_t c) {
#pragma unroll
  for (int i = 0; i < 4; ++i) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[i], c, 0, 0, 0);
  return c;
}

// NB = DP / 16 column blocks of the keys.  One workgroup (4 waves) per (head, chunk, sequence).
template <int NB>
__global__ void __launch_bounds__(256) delta_chunk_prepare_kernel(DeltaParams p) {
  constexpr int DP = NB * 16, KS = DP + 4, AS = CH + 4;   // LDS row strides (floats)
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float* kt = sm;                       // [64][KS] keys
  float* am = kt + CH * KS;             // [64][AS] A, later the inverted diagonal blocks in place
  __shared__ double gd[CH];
  __shared__ float beta[CH], eg[CH];
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, lr = lane & 15, lq = lane >> 4;
  const int h = blockIdx.x, ch = blockIdx.y, b = blockIdx.z, H = p.H, G = p.G, V = p.V, g = h / (H / G);
  const int len = p.lens ? min(p.lens[b], p.T) : p.T;
  const int n = min(CH, len - ch * CH);
  if (n <= 0) return;
  const int64_t m0 = (int64_t)b * p.T + ch * CH;
  const int64_t cell = ((int64_t)b * p.nch + ch) * H + h;

  const int64_t qkcell = (((int64_t)b * p.nch + ch) * G + g) * CH * DP;
  for (int i = tid; i < CH * (DP / 4); i += 256) {   // block (d / 16, t / 16), lane i % 64: column d, four tokens
    const int d = 16 * (i / 256) + (i & 15), t = 16 * ((i / 64) & 3) + 4 * ((i / 16) & 3);
    const f32x4_t v = ld4(p.kn + qkcell + 4 * i);
#pragma unroll
    for (int e = 0; e < 4; ++e) kt[(t + e) * KS + d] = v[e];
  }
  if (w == 0) {
    double s = lane < n ? (double)p.lg[(m0 + lane) * H + h] : 0.0;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const double q = __shfl_up(s, o, 64);
      if (lane >= o) s += q;
    }
    gd[lane] = s;
    eg[lane] = expf((float)s);
    beta[lane] = lane < n ? p.beta[(m0 + lane) * H + h] : 0.f;
    const double last = __shfl(s, 63, 64);
    float* e = p.ceg + cell * (2 * CH);
    e[lane] = expf((float)s);                  // e^G
    e[CH + lane] = expf((float)(last - s));    // e^(G_C - G)
  }
  __syncthreads();

  // ---- the 10 lower blocks of K K^T and of Q K^T, five products a wave
  float* P = p.cp + cell * (CH * CH);
  for (int job = w; job < 20; job += 4) {
    const bool isq = job >= 10;
    int bi = 0, bj = isq ? job - 10 : job;
    while (bj > bi) bj -= ++bi;               // (0,0) (1,0) (1,1) (2,0) ...
    const int t = 16 * bi + lr;
    f32x4_t acc = {0.f, 0.f, 0.f, 0.f}, acc2 = acc;
#pragma unroll
    for (int kb = 0; kb < NB; ++kb) {
      f32x4_t a;
      if (isq) a = ld4(p.qn + qkcell + ((bi * NB + kb) * 64 + lane) * 4);
      else a = ld4(kt + t * KS + 16 * kb + 4 * lq);
      const f32x4_t bb = ld4(kt + (16 * bj + lr) * KS + 16 * kb + 4 * lq);
      if (kb & 1) acc2 = mma4(a, bb, acc2);
      else acc = mma4(a, bb, acc);
    }
    acc += acc2;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int row = 16 * bi + 4 * lq + i, col = 16 * bj + lr;
      const bool in = isq ? col <= row : col < row;
      const float v = in ? acc[i] * expf((float)(gd[row] - gd[col])) : 0.f;
      if (isq) P[((bi * 4 + bj) * 64 + (lr / 4) * 16 + 4 * lq + i) * 4 + (lr & 3)] = v;
      else am[row * AS + col] = v * beta[row];
    }
  }
  __syncthreads();

  // ---- diagonal block w: (I + A_ww)^-1, column lr by the 16 lanes of the first quarter
  {
    float x[16];
    const float* a = am + (16 * w) * AS + 16 * w;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float s = i == lr ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < i; ++j) s -= a[i * AS + j] * x[j];
      x[i] = s;
    }
    __builtin_amdgcn_wave_barrier();
    if (lq == 0) {
#pragma unroll
      for (int i = 0; i < 16; ++i) am[(16 * w + i) * AS + 16 * w + lr] = x[i];
    }
  }
  __syncthreads();

  // ---- (I + A) [Y | W] = diag(beta) [V | e^G K], 16 columns at a time; a wave takes every fourth
  const int nv = (V + 15) / 16;
  for (int ct = w; ct < nv + NB; ct += 4) {
    const bool isv = ct < nv;
    const int col = (isv ? ct : ct - nv) * 16 + lr;
    f32x4_t y[4];
#pragma unroll
    for (int bi = 0; bi < 4; ++bi) {
      f32x4_t r;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = 16 * bi + 4 * lq + i;
        float v;
        if (isv) v = t < n && col < V ? p.vn[((m0 + t) * H + h) * V + col] : 0.f;
        else v = kt[t * KS + col] * eg[t];
        r[i] = v * beta[t];
      }
      f32x4_t s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int bk = 0; bk < bi; ++bk) s = mma4(ld4(am + (16 * bi + lr) * AS + 16 * bk + 4 * lq), y[bk], s);
      r -= s;
      y[bi] = mma4(ld4(am + (16 * bi + lr) * AS + 16 * bi + 4 * lq), r, f32x4_t{0.f, 0.f, 0.f, 0.f});
    }
#pragma unroll
    for (int bi = 0; bi < 4; ++bi) {
      if (isv) {
        st4(p.cy + ((cell * nv + ct) * 4 + bi) * 256 + lane * 4, y[bi]);
      } else {
        float* o = p.cw + (cell * 4 + bi) * (NB * 256) + (ct - nv) * 256;
#pragma unroll
        for (int i = 0; i < 4; ++i) o[((lr / 4) * 16 + 4 * lq + i) * 4 + (lr & 3)] = y[bi][i];
      }
    }
  }
}

// 16 state columns of one head, 8 waves.  Waves 0-3 (tokens 16 w .. of a chunk) compute U, waves 4-7 the
// outputs of the same tokens; the state's row blocks are spread over all of them.  So every SIMD has one
// wave on the chain state -> U -> state and one whose work fills its waits.  Operands are fetched two
// chunks ahead into two register sets.
template <typename T, int NB>
__global__ void __launch_bounds__(512, 2) delta_chunk_scan_kernel(DeltaParams p) {
  constexpr int DP = NB * 16, TPW = (NB + 7) / 8;
  __shared__ __attribute__((aligned(16))) f32x4_t ss[NB][64], us[4][64], ud[4][64];
  const int tid = threadIdx.x, lane = tid & 63, w8 = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lq = lane >> 4;
  const int w = w8 & 3;
  const bool outw = w8 >= 4;
  const int bh = blockIdx.x % (p.B * p.H), v0 = (blockIdx.x / (p.B * p.H)) * 16;   // a head's columns on one XCD
  const int b = bh / p.H, h = bh % p.H, H = p.H, G = p.G, V = p.V, g = h / (H / G);
  const int len = p.lens ? min(p.lens[b], p.T) : p.T;
  if (len <= 0) return;
  const int slot = slot_of(p.slots, b, p.nslots);
  const int64_t p0 = pos_of(p.pos, p.pos_stride, b);
  const int v = v0 + lr;
  const bool vok = v < V;
  float* state = p.state + (((int64_t)slot * H + h) * V + min(v, V - 1)) * DP;
  f32x4_t S[TPW];
#pragma unroll
  for (int i = 0; i < TPW; ++i) {
    const int rt = w8 + 8 * i;
    S[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    if (rt < NB) {
      if (p0 > 0) S[i] = ld4(state + rt * 16 + 4 * lq);
      ss[rt][lane] = S[i];
    }
  }
  const int nch = (len + CH - 1) / CH;
  const f32x4_t zero = {0.f, 0.f, 0.f, 0.f};
  // one chunk's operands: rows of W (U waves) or of Q (output waves), K^T for the own state blocks, the
  // Y tile (U waves) or the P rows (output waves), e^G / e^(G_C - G) of the own rows and e^(G_C).  What a
  // padded token brings is zero.
  struct Ops {
    f32x4_t rowf[NB], kf[TPW][4], pf[4], eg;
    float ec;
  };
  Ops set[2];
  const int nv = (V + 15) / 16;
  // (past the last chunk the last one is read again: an unconditional fetch keeps the number of loads in
  // flight known, so a wait covers exactly one set)
  auto fetch = [&](int c, Ops& o) {
    c = min(c, nch - 1);
    const int64_t cell = ((int64_t)b * p.nch + c) * H + h, qkcell = (((int64_t)b * p.nch + c) * G + g) * CH * DP;
    const float* s = (outw ? p.qn + qkcell : p.cw + cell * CH * DP) + w * (NB * 256) + lane * 4;
#pragma unroll
    for (int kb = 0; kb < NB; ++kb) o.rowf[kb] = ld4(s + kb * 256);
    const float* e = p.ceg + cell * (2 * CH);
    o.eg = ld4(e + (outw ? 0 : CH) + 16 * w + 4 * lq);
    o.ec = e[CH - 1];
    // (output waves use the blocks up to the diagonal, the U waves the first)
    const float* q = outw ? p.cp + cell * (CH * CH) + w * 1024 + lane * 4 : p.cy + ((cell * nv + v0 / 16) * 4 + w) * 256 + lane * 4;
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) o.pf[kb] = ld4(q + (outw ? kb * 256 : 0));
    const float* k = p.kn + qkcell + lane * 4;
#pragma unroll
    for (int j = 0; j < TPW; ++j)
#pragma unroll
      for (int kb = 0; kb < 4; ++kb) o.kf[j][kb] = ld4(k + ((8 * j + 8 <= NB ? w8 + 8 * j : min(w8 + 8 * j, NB - 1)) * 4 + kb) * 256);
  };
  fetch(0, set[0]);
  asm volatile("" ::: "memory");   // (not interleaved: the loop's waits count on the order)
  fetch(1, set[1]);
  lds_barrier();
  auto chunk = [&](int c, Ops& o) {
    f32x4_t a0 = zero, a1 = zero, sb[NB];
#pragma unroll
    for (int kb = 0; kb < NB; ++kb) sb[kb] = ss[kb][lane];
    __builtin_amdgcn_sched_barrier(0);   // all reads in flight before the first product
#pragma unroll
    for (int kb = 0; kb < NB; kb += 2) {   // NB is even
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.rowf[kb][i], sb[kb][i], a0, 0, 0, 0);
        a1 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.rowf[kb + 1][i], sb[kb + 1][i], a1, 0, 0, 0);
      }
    }
    f32x4_t r = a0 + a1;   // W S or Q S
    if (!outw) {
      r = o.pf[0] - r;
      us[w][lane] = r;
      ud[w][lane] = r * o.eg;
    }
    lds_barrier();
    f32x4_t ub[4];
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) ub[kb] = ud[kb][lane];
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int j = 0; j < TPW; ++j) {
      if (8 * j + 8 <= NB || w8 + 8 * j < NB) {
        f32x4_t x = S[j] * o.ec, y = zero;
#pragma unroll
        for (int kb = 0; kb < 4; kb += 2) {
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            x = __builtin_amdgcn_mfma_f32_16x16x4f32(o.kf[j][kb][i], ub[kb][i], x, 0, 0, 0);
            y = __builtin_amdgcn_mfma_f32_16x16x4f32(o.kf[j][kb + 1][i], ub[kb + 1][i], y, 0, 0, 0);
          }
        }
        S[j] = x + y;
        ss[w8 + 8 * j][lane] = S[j];
      }
    }
    if (outw) {
      r *= o.eg;
#pragma unroll
      for (int kb = 0; kb < 4; ++kb)
        if (kb <= w) r = mma4(o.pf[kb], us[kb][lane], r);
#pragma unroll
      for (int i = 0; i < 4; ++i) {   // (a wave of padded tokens stores nothing)
        const int t = c * CH + 16 * w + 4 * lq + i;
        if (vok && t < len) p.o[(((int64_t)b * p.T + t) * H + h) * V + v] = r[i];
      }
    }
    fetch(c + 2, o);
    lds_barrier();
  };
  int c = 0;
  for (; c + 1 < nch; c += 2) {
    chunk(c, set[0]);
    chunk(c + 1, set[1]);
  }
  if (c < nch) chunk(c, set[0]);
  if (vok) {
#pragma unroll
    for (int i = 0; i < TPW; ++i)
      if (w8 + 8 * i < NB) st4(state + (w8 + 8 * i) * 16 + 4 * lq, S[i]);
  }
  if (v0 == 0 && h == 0) ring_write<T>(p, b, slot, p0, len, tid, 512);
}

template <typename T, int NB>
static int run_chunk(const DeltaParams& p, hipStream_t s) {
  const size_t lds = (size_t)CH * (NB * 16 + 4 + CH + 4) * 4;
  static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(&delta_chunk_prepare_kernel<NB>),
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
  if (attr != hipSuccess) return 2;
  hipLaunchKernelGGL((delta_chunk_prepare_kernel<NB>), dim3((unsigned)p.H, (unsigned)p.nch, (unsigned)p.B), dim3(256), lds, s, p);
  if (hipGetLastError() != hipSuccess) return 1;
  const int64_t grid = (int64_t)ceil_div(p.V, 16) * p.B * p.H;
  hipLaunchKernelGGL((delta_chunk_scan_kernel<T, NB>), dim3((unsigned)grid), dim3(512), 0, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

template <typename T>
static int dispatch_chunk(const DeltaParams& p, hipStream_t s) {
  switch (p.DP / 32) {
    case 1: return run_chunk<T, 2>(p, s);
    case 2: return run_chunk<T, 4>(p, s);
    case 3: return run_chunk<T, 6>(p, s);
    case 4: return run_chunk<T, 8>(p, s);
    case 5: return run_chunk<T, 10>(p, s);
    case 6: return run_chunk<T, 12>(p, s);
    case 7: return run_chunk<T, 14>(p, s);
    case 8: return run_chunk<T, 16>(p, s);
  }
  return -1;
}

}  // namespace hybrid

int delta_chunk_launch(bool f32, const DeltaParams& p, hipStream_t s) {
  return f32 ? hybrid::dispatch_chunk<float>(p, s) : hybrid::dispatch_chunk<uint16_t>(p, s);
}

}  // namespace nxd
