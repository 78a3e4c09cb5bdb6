// Parameters of the residual sum + grouped RMS norms (csrc/hybrid/group_norm.hip).
#pragma once
#include "hybrid.h"

namespace nxd {

struct GroupNormParams {
  int64_t M, R;            // rows of x, rows of h
  int W, groups;
  float* x;                // [M, W]
  const void* embed;       // [vocab, W] (nullable)
  const int64_t* ids;      // [M]
  int64_t vocab;
  const void* add[2];      // [M, ld_add] (nullable)
  int64_t ld_add[2];
  const void* pairs;       // [npairs, W] (nullable)
  const int* inverse;      // [M, k] (nullable: row m k + j)
  int npairs, k;
  const float* w[2];       // [W]
  void* h[2];              // [R, ldh] (nullable)
  int64_t ldh;
  float eps;
  const int64_t* rows;     // [R] (nullable: all)
  bool store;
};

}  // namespace nxd
