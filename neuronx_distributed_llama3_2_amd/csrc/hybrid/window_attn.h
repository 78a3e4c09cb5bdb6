// Parameters of the windowed, differential and pooled-block attention kernels (csrc/hybrid/window_attn*.hip,
// pooled_attn.hip).
#pragma once
#include "hybrid.h"

namespace nxd {

struct WindowAttnParams {
  int B, T;               // sequences, new tokens per sequence (row b * T + t)
  int H, G, maps, D, V;   // query heads, key/value heads, maps per head (1: plain, 2: differential), sizes
  void* buf;              // [B T, ldb]: q (H maps D) | k (G maps D) | v (G V), activation type
  int64_t ldb;
  // keys and values of the step's tokens, row b * T + t: [.., ldk], [.., ldv]
  const void *kbuf, *vbuf;
  int64_t ldk, ldv;
  int v_off;              // column of the first value in a row of buf
  const int64_t* pos;     // position of each sequence's first new token: pos[b * pos_stride]
  int64_t pos_stride;
  const int* lens;        // [B] valid new tokens (nullable: T)
  const int* slots;       // [B] cache slots (nullable: identity)
  int nslots;
  void* kc;               // [slots, G maps, cap, D] ring by position: p in entry p % cap
  void* vc;               // [slots, G, cap, V]
  int cap;
  // qkv preparation
  const float* bias;      // [H maps D + G maps D + G V] (nullable)
  const float *qn_w, *kn_w;   // [D] (nullable: no norm), norm_all: [H D] and [G D]
  bool norm_all;          // one norm over all heads of the row
  float eps;
  const float *cos_t, *sin_t; // [max_pos, rot / 2]
  int rot, max_pos;
  // attention
  float scale, softcap;   // softcap <= 0: none
  int window;             // <= 0: all earlier tokens
  float lam, out_scale, out_eps;   // differential: (a1 - lam a2) / rms * out_scale; one map: a * out_scale
  void* y;                // [B T, ldy] heads side by side
  int64_t ldy;
  int from_buf;           // keys of this step's buffer (prompt from position 0) instead of the cache
  // pooled blocks (pool > 0): of `pool` tokens each, a query at i sees those that end at i - window or before
  int pool, pcap;         // tokens of a block, entries of the pooled caches
  void *pk, *pv;          // [slots, G, pcap, D], [slots, G, pcap, V]: means of a block's keys and values
  // split decode
  int share;              // query heads of a workgroup (of one key / value head)
  int splits, tiles;      // workgroups per (sequence, heads), 64-key tiles each
  float* part;            // [B H, splits, maps (V + 2)] partial sums (splits > 1)
  int* tickets;           // [B H] arrivals, zero between launches (splits > 1)
};

namespace hybrid {

// pooled blocks that the query at position ps sees
__device__ __forceinline__ int blocks_seen(const WindowAttnParams& p, int64_t ps) {
  const int64_t n = ps - p.window + 1;
  return n > 0 ? (int)min(n / p.pool, (int64_t)p.pcap) : 0;
}

}  // namespace hybrid
}  // namespace nxd
