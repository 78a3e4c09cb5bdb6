// Prompt attention of one or two maps per head on the matrix cores (bf16, causal, optional window and
// score cap): the body shared by the per-size translation units window_attn_prompt_*.hip.
//
//   * workgroup = 128 query rows of one (sequence, head); 4 waves a map, 32 rows each, the query
//     fragments stay in registers.  The maps of a row are in different waves: the softmax of a capped
//     score costs three transcendental instructions, far more time than its share of the products,
//     so what counts is two waves per SIMD with few registers each, not reading V once for both maps;
//   * tiles of 64 keys (K of every map, V once) go global -> registers -> LDS one tile ahead of their
//     use, into two buffers; head sizes are padded to the fragment size with zeros in LDS, rows are
//     16 bytes longer than their data so that row reads spread over the banks;
//   * S^T = K Q^T (v_mfma_f32_32x32x16_bf16): a lane holds 16 scores of one query, so the softmax is
//     lane-local plus one cross-half exchange and P^T is the B operand of O^T += V^T P^T directly;
//   * with a score cap of at most 40 the maximum is known in advance, exp(cap tanh(x) - cap) is
//     computed as exp(-2 cap / (exp(2 x) + 1)) and there is no running maximum to follow;
//   * POOL (one map): the tiles of the pooled blocks that some row sees come first, read from the pooled
//     cache, in the same softmax;
//   * at the end the second map's waves hand their rows to the first's through LDS: the difference, its
//     RMS over the head and the output scale are applied there in fp32.
#pragma once
#include "window_attn.h"

namespace nxd {
namespace hybrid {

constexpr float kLog2e = 1.4426950408889634f;

typedef __attribute__((address_space(3))) char lds_char_t;
__device__ __forceinline__ uint32_t lds_addr(const char* ptr) { return (uint32_t)(uintptr_t)(const lds_char_t*)ptr; }
__device__ __forceinline__ float pair_sum(float x) {   // lanes l and l ^ 32
  const auto pr = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
  return __uint_as_float(pr[0]) + __uint_as_float(pr[1]);
}
__device__ __forceinline__ float pair_max(float x) {
  const auto pr = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
  return fmaxf(__uint_as_float(pr[0]), __uint_as_float(pr[1]));
}

// N ds_read_b64_tr_b16 results may be used after this (those issued later stay in flight)
template <int N, int LATER>
__device__ __forceinline__ void tr_wait(short4_t (&v)[N]) {
  asm volatile("s_waitcnt lgkmcnt(%1)" : "+v"(v[0]) : "n"(LATER <= 15 ? LATER : 15));
#pragma unroll
  for (int i = 1; i < N; ++i) asm volatile("" : "+v"(v[i]));
}

// KS 16-wide steps of the (padded) query size, NDB 32-wide blocks of the (padded) value size; FIXED: the
// scores' maximum is the cap (0 < softcap <= 40), else a running maximum is kept
template <int KS, int NDB, int MAPS, bool FIXED, bool POOL = false>
__global__ void __launch_bounds__(256 * MAPS, 2) attn_prompt_kernel(WindowAttnParams p) {
  constexpr int BN = 64, DP = KS * 16, VP = NDB * 32, NT = 256 * MAPS;
  constexpr int KROW = DP * 2 + 16, VROW = VP * 2 + 16;         // bytes of an LDS row
  constexpr int KTILE = BN * KROW, VTILE = BN * VROW, BUF = MAPS * KTILE + VTILE;
  constexpr int KCH = DP / 8, VCH = VP / 8;                     // 16-byte chunks of a row
  constexpr int NK = (MAPS * BN * KCH + NT - 1) / NT, NV = (BN * VCH + NT - 1) / NT;
  extern __shared__ __attribute__((aligned(16))) char smem[];

  const int nq = (p.T + 127) / 128;
  const int bh = blockIdx.x % (p.B * p.H), mblk = nq - 1 - (int)blockIdx.x / (p.B * p.H);
  const int b = bh / p.H, h = bh % p.H, g = h / (p.H / p.G);
  const int tid = threadIdx.x, lane = tid & 63, w = (tid >> 6) & 3, r = lane & 31, hh = lane >> 5;
  const int c = MAPS == 1 ? 0 : __builtin_amdgcn_readfirstlane(tid >> 8);   // this wave's map
  const int len = p.lens ? min(p.lens[b], p.T) : p.T;
  const int qb0 = mblk * 128, q0 = qb0 + w * 32, my_q = q0 + r;
  uint16_t* yrow = static_cast<uint16_t*>(p.y) + ((int64_t)b * p.T + min(my_q, p.T - 1)) * p.ldy + (int64_t)h * p.V;
  if (qb0 >= len) {   // padding only: defined values for the projection that follows
    if (my_q < p.T && c == 0)
      for (int d = hh * 4; d < p.V; d += 8) *reinterpret_cast<u32x2_t*>(yrow + d) = u32x2_t{0u, 0u};
    return;
  }
  const uint16_t* base = static_cast<const uint16_t*>(p.buf) + (int64_t)b * p.T * p.ldb;
  const uint16_t* qrow = base + (int64_t)min(my_q, p.T - 1) * p.ldb + ((int64_t)h * MAPS + c) * p.D;
  const uint16_t* kb = static_cast<const uint16_t*>(p.kbuf) + (int64_t)b * p.T * p.ldk + (int64_t)g * MAPS * p.D;
  const uint16_t* vb = static_cast<const uint16_t*>(p.vbuf) + (int64_t)b * p.T * p.ldv + (int64_t)g * p.V;
  const int64_t phead = POOL ? (int64_t)slot_of(p.slots, b, p.nslots) * p.G + g : 0;
  const uint16_t* pkb = static_cast<const uint16_t*>(p.pk) + phead * p.pcap * p.D;
  const uint16_t* pvb = static_cast<const uint16_t*>(p.pv) + phead * p.pcap * p.V;

  bf16x8_t qf[KS];
#pragma unroll
  for (int s = 0; s < KS; ++s) {
    const int d = 16 * s + 8 * hh;
    u32x4_t v = {0u, 0u, 0u, 0u};
    if (d < p.D) v = *reinterpret_cast<const u32x4_t*>(qrow + d);
    qf[s] = __builtin_bit_cast(bf16x8_t, v);
  }

  const int kend = min(len, qb0 + 128);
  const int kbeg = p.window > 0 ? max(0, qb0 - p.window + 1) / BN * BN : 0;
  const int pend = POOL ? blocks_seen(p, kend - 1) : 0;                    // pooled blocks some row of the workgroup sees
  const int my_blocks = POOL ? blocks_seen(p, my_q) : 0;
  const int first_blocks = POOL ? blocks_seen(p, q0) : 0, last_blocks = POOL ? blocks_seen(p, q0 + 31) : 0;   // of the wave
  const int wave_lo = p.window > 0 ? q0 - p.window + 1 : 0, wave_hi = q0 + 31;   // keys some row may see

  // staging registers of the next tile
  u32x4_t kst[NK], vst[NV];
  auto fetch = [&](int k0, bool pooled) {
    const uint16_t *ksrc = POOL && pooled ? pkb : kb, *vsrc = POOL && pooled ? pvb : vb;
    const int64_t lk = POOL && pooled ? p.D : p.ldk, lv = POOL && pooled ? p.V : p.ldv;
    const int last = (POOL && pooled ? pend : len) - 1;
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int e = tid + NT * i, ch = e % KCH, row = (e / KCH) % BN, m = e / (KCH * BN);
      kst[i] = u32x4_t{0u, 0u, 0u, 0u};
      if (m < MAPS && ch * 8 < p.D)
        kst[i] = *reinterpret_cast<const u32x4_t*>(ksrc + (int64_t)min(k0 + row, last) * lk + m * p.D + ch * 8);
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int e = tid + NT * i, ch = e % VCH, row = e / VCH;
      vst[i] = u32x4_t{0u, 0u, 0u, 0u};
      if (row < BN && ch * 8 < p.V)
        vst[i] = *reinterpret_cast<const u32x4_t*>(vsrc + (int64_t)min(k0 + row, last) * lv + ch * 8);
    }
  };
  auto stash = [&](int buf) {
    char* kl = smem + buf * BUF;
    char* vl = kl + MAPS * KTILE;
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int e = tid + NT * i, ch = e % KCH, row = e / KCH;   // row runs over the maps' tiles
      if (row < MAPS * BN) *reinterpret_cast<u32x4_t*>(kl + row * KROW + ch * 16) = kst[i];
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int e = tid + NT * i, ch = e % VCH, row = e / VCH;
      if (row < BN) *reinterpret_cast<u32x4_t*>(vl + row * VROW + ch * 16) = vst[i];
    }
  };

  f32x16_t acc[NDB];
  float mx = -INFINITY, ls = 0.f;
#pragma unroll
  for (int i = 0; i < NDB; ++i) acc[i] = f32x16_t{0};
  constexpr int DBG = NDB < 4 ? NDB : 4, NG = 4 * (NDB / DBG);   // V blocks of a read group, groups of a tile
  static_assert(NDB % DBG == 0, "whole read groups");
  const float cap_in = p.softcap > 0.f ? 2.f * p.scale / p.softcap * kLog2e : 0.f;   // exp2(cap_in s) = exp(2 x)
  const float cap_out = 2.f * p.softcap * kLog2e;

  // transposed V reads: a group of 16 lanes covers 4 keys x 16 columns
  const int gi = lane & 15, tq = gi >> 2, tp = gi & 3, grp = lane >> 4;
  const uint32_t vlane = lds_addr(smem) + MAPS * KTILE + (uint32_t)((4 * hh + tq) * VROW + (16 * (grp & 1) + 4 * tp) * 2);

  bool pooled = pend > 0;   // tiles of pooled blocks first
  int k0 = pooled ? 0 : kbeg;
  fetch(k0, pooled);
  stash(0);
  __syncthreads();
  int buf = 0;
  for (;; buf ^= 1) {
    const bool nextp = POOL && pooled && k0 + BN < pend;
    const int knext = POOL && pooled && !nextp ? kbeg : k0 + BN;
    const bool more = nextp || knext < kend;
    if (more) fetch(knext, nextp);
    if (POOL && pooled ? k0 < last_blocks : (k0 <= wave_hi && k0 + BN - 1 >= wave_lo)) {
      const char* kl = smem + buf * BUF + c * KTILE;
      const uint32_t va = vlane + buf * BUF;
      const bool edge = POOL && pooled ? k0 + BN > first_blocks
                                       : k0 + BN - 1 > q0 || (p.window > 0 && k0 < q0 + 31 - p.window + 1);
      f32x16_t s[2];
      s[0] = f32x16_t{0};
      s[1] = f32x16_t{0};
#pragma unroll
      for (int st = 0; st < KS; ++st)
#pragma unroll
        for (int j = 0; j < 2; ++j) {
          const u32x4_t kf = *reinterpret_cast<const u32x4_t*>(kl + (32 * j + r) * KROW + (2 * st + hh) * 16);
          s[j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, kf), qf[st], s[j], 0, 0, 0);
        }
      // O^T += V^T P^T, 16 keys at a time: a lane's 8 keys are 16 q + 4 hh .. + 3 and those + 8
      short4_t vt[2][2 * DBG];
      auto issue = [&](int grp_, short4_t (&v)[2 * DBG]) {   // group: keys 16 (grp / (NDB / DBG)), blocks DBG (grp % ..)
        const uint32_t a = va + (grp_ / (NDB / DBG)) * 16 * VROW + (grp_ % (NDB / DBG)) * DBG * 64;
#pragma unroll
        for (int db = 0; db < DBG; ++db) {
          asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(v[2 * db]) : "v"(a), "n"(64 * db));
          asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(v[2 * db + 1]) : "v"(a), "n"(64 * db + 8 * VROW));
        }
      };
      issue(0, vt[0]);
      // element e of s[j] is key k0 + 32 j + (e & 3) + 8 (e >> 2) + 4 hh
      const int hi = (POOL && pooled ? my_blocks - 1 : my_q) - k0 - 4 * hh;           // seen: offset <= hi
      const int lo = p.window > 0 && !(POOL && pooled) ? my_q - p.window + 1 - k0 - 4 * hh : -0x40000000;  // and >= lo
      float sum = 0.f;
      bf16x8_t pf[4];
      if constexpr (FIXED) {
#pragma unroll
        for (int j = 0; j < 2; ++j)
#pragma unroll
          for (int e = 0; e < 16; ++e)
            s[j][e] = __builtin_amdgcn_exp2f(-cap_out * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(s[j][e] * cap_in) + 1.f));
        if (edge) {
#pragma unroll
          for (int j = 0; j < 2; ++j)
#pragma unroll
            for (int e = 0; e < 16; ++e) {
              const int o = 32 * j + (e & 3) + 8 * (e >> 2);
              s[j][e] = o <= hi && o >= lo ? s[j][e] : 0.f;
            }
        }
#pragma unroll
        for (int j = 0; j < 2; ++j)
#pragma unroll
          for (int e = 0; e < 16; ++e) {
            sum += s[j][e];
            pf[2 * j + (e >> 3)][e & 7] = (__bf16)s[j][e];
          }
      } else {
        if (p.softcap > 0.f) {
#pragma unroll
          for (int j = 0; j < 2; ++j)
#pragma unroll
            for (int e = 0; e < 16; ++e)   // log2(e) cap tanh(x)
              s[j][e] = cap_out * (0.5f - __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(s[j][e] * cap_in) + 1.f));
        } else {
          s[0] *= p.scale * kLog2e;
          s[1] *= p.scale * kLog2e;
        }
        if (edge) {
#pragma unroll
          for (int j = 0; j < 2; ++j)
#pragma unroll
            for (int e = 0; e < 16; ++e) {
              const int o = 32 * j + (e & 3) + 8 * (e >> 2);
              s[j][e] = o <= hi && o >= lo ? s[j][e] : -INFINITY;
            }
        }
        float tmax = -INFINITY;
#pragma unroll
        for (int j = 0; j < 2; ++j)
#pragma unroll
          for (int e = 0; e < 16; ++e) tmax = fmaxf(tmax, s[j][e]);
        tmax = pair_max(tmax);
        if (tmax > mx) {
          const float f = __builtin_amdgcn_exp2f(mx - tmax);   // first tile: exp2(-inf) = 0
          mx = tmax;
          ls *= f;
#pragma unroll
          for (int i = 0; i < NDB; ++i) acc[i] *= f;
        }
        const float m = mx == -INFINITY ? 0.f : mx;
#pragma unroll
        for (int j = 0; j < 2; ++j)
#pragma unroll
          for (int e = 0; e < 16; ++e) {
            const float pv = __builtin_amdgcn_exp2f(s[j][e] - m);
            sum += pv;
            pf[2 * j + (e >> 3)][e & 7] = (__bf16)pv;
          }
      }
      ls += pair_sum(sum);
#pragma unroll
      for (int q = 0; q < NG; ++q) {
        if (q + 1 < NG) {
          issue(q + 1, vt[(q + 1) & 1]);
          tr_wait<2 * DBG, 2 * DBG>(vt[q & 1]);
        } else {
          tr_wait<2 * DBG, 0>(vt[q & 1]);
        }
#pragma unroll
        for (int i = 0; i < DBG; ++i) {
          const int db = (q % (NDB / DBG)) * DBG + i;
          const short4_t lo4 = vt[q & 1][2 * i], hi4 = vt[q & 1][2 * i + 1];
          const short __attribute__((ext_vector_type(8))) a8 = {lo4[0], lo4[1], lo4[2], lo4[3], hi4[0], hi4[1], hi4[2], hi4[3]};
          acc[db] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, a8), pf[q / (NDB / DBG)], acc[db], 0, 0, 0);
        }
      }
    }
    if (!more) break;
    stash(buf ^ 1);
    lds_barrier();
    k0 = knext;
    pooled = nextp;
  }

  const bool live = my_q < len;
  const float inv = live && ls > 0.f ? 1.f / ls : 0.f;
#pragma unroll
  for (int db = 0; db < NDB; ++db) acc[db] *= inv;
  float sc = p.out_scale;
  if constexpr (MAPS == 2) {
    __syncthreads();   // (the tiles' last readers are done)
    float* xch = reinterpret_cast<float*>(smem) + w * (NDB * 16 * 64) + lane;   // [wave][element][lane]
    if (c == 1) {
#pragma unroll
      for (int db = 0; db < NDB; ++db)
#pragma unroll
        for (int e = 0; e < 16; ++e) xch[(db * 16 + e) * 64] = acc[db][e];
    }
    __syncthreads();
    if (c == 1) return;
    float ss = 0.f;
#pragma unroll
    for (int db = 0; db < NDB; ++db)
#pragma unroll
      for (int e = 0; e < 16; ++e) {
        acc[db][e] -= p.lam * xch[(db * 16 + e) * 64];
        ss += acc[db][e] * acc[db][e];   // padded columns are zero
      }
    sc = p.out_scale / sqrtf(pair_sum(ss) / (float)p.V + p.out_eps);
  }
  if (my_q >= p.T) return;
#pragma unroll
  for (int db = 0; db < NDB; ++db)
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const int d = 32 * db + 8 * q + 4 * hh;
      if (d < p.V)
        *reinterpret_cast<u32x2_t*>(yrow + d) =
            u32x2_t{pack2bf(acc[db][4 * q] * sc, acc[db][4 * q + 1] * sc),
                    pack2bf(acc[db][4 * q + 2] * sc, acc[db][4 * q + 3] * sc)};
    }
}

template <int KS, int NDB, int MAPS, bool FIXED, bool POOL = false>
int attn_prompt_run(const WindowAttnParams& p, hipStream_t s) {
  constexpr size_t tiles = 2 * (size_t)64 * (MAPS * (KS * 32 + 16) + NDB * 64 + 16);
  constexpr size_t xch = MAPS == 2 ? (size_t)4 * NDB * 16 * 64 * 4 : 0;
  constexpr size_t lds = tiles > xch ? tiles : xch;
  static_assert(lds <= 160 * 1024, "LDS of a compute unit");
  static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(&attn_prompt_kernel<KS, NDB, MAPS, FIXED, POOL>),
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
  if (attr != hipSuccess) return 2;
  const int64_t grid = (int64_t)((p.T + 127) / 128) * p.B * p.H;
  hipLaunchKernelGGL((attn_prompt_kernel<KS, NDB, MAPS, FIXED, POOL>), dim3((unsigned)grid), dim3(256 * MAPS), lds, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

// pooled blocks: values are as wide as keys
template <int KS>
int attn_prompt_pooled(const WindowAttnParams& p, hipStream_t s) {
  if (p.maps != 1 || p.V > KS * 16) return -1;
  return attn_prompt_run<KS, (KS * 16 + 31) / 32, 1, false, true>(p, s);
}

template <int KS, int MAPS, bool FIXED>
int attn_prompt_by_v(const WindowAttnParams& p, hipStream_t s) {
  if (p.V <= 32) return attn_prompt_run<KS, 1, MAPS, FIXED>(p, s);
  if (p.V <= 64) return attn_prompt_run<KS, 2, MAPS, FIXED>(p, s);
  if (p.V <= 96) return attn_prompt_run<KS, 3, MAPS, FIXED>(p, s);
  if (p.V <= 128) return attn_prompt_run<KS, 4, MAPS, FIXED>(p, s);
  return attn_prompt_run<KS, 8, MAPS, FIXED>(p, s);
}

}  // namespace hybrid
}  // namespace nxd
