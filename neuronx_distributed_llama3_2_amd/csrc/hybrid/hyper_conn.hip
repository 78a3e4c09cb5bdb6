// Hyper-connections: S residual streams instead of one, mixed around every sublayer.
//
//   u   = sum_s read[s] x_s                      (the sublayer's input, then a zero-centred RMSNorm)
//   x_t = sum_s mix[s][t] x_s + write[t] (y + bias)   (from the old streams, after the sublayer)
//
// One launch between two sublayers does the write of the one and the read + norm of the next: a row's
// streams are read once and written once (fp32, [M, S, W]), y is the only other large operand.  The
// first launch of a forward takes its rows from the embedding table (every stream starts as the token's
// embedding), the last one reads with all-ones weights (the sum of the streams) and the model's norm.
#include "hybrid.h"

namespace nxd {
namespace hybrid {

struct HyperParams {
  float* x;              // [M, S, W] streams, updated in place
  const void* embed;     // [V, W] (activation type): rows gathered instead of x
  const int64_t* ids;    // [M]
  int64_t vocab;
  const void* y;         // [M, W] sublayer output (nullable: streams pass through)
  int64_t ldy;
  const float* bias;     // [W] added to y (nullable)
  const float* mix;      // [S, S] (from, to)
  const float* write;    // [S]
  const float* read;     // [S] (nullable: no norm output)
  const float* norm_w;   // [W] stored around zero
  float eps;
  void* h;               // [R, W] normalised input of the next sublayer (activation type)
  int64_t ldh;
  const int64_t* rows;   // [R] rows of x (nullable: identity)
  int store;             // write the streams back
  int W;
};

template <typename T, int S, int V>
__global__ void __launch_bounds__(256) hyper_step_kernel(HyperParams p) {
  extern __shared__ __attribute__((aligned(16))) float us[];   // [W]
  __shared__ float red[16];
  const int64_t row = p.rows ? p.rows[blockIdx.x] : (int64_t)blockIdx.x;
  const int tid = threadIdx.x, W = p.W;
  float* xr = p.x + row * S * W;
  const T* er = nullptr;
  if (p.embed) {
    const int64_t id = p.ids[row];
    if (id >= 0 && id < p.vocab) er = static_cast<const T*>(p.embed) + id * W;   // else: a zero row
  }
  float mix[S * S], wr[S], rd[S];
#pragma unroll
  for (int i = 0; i < S; ++i) {
    wr[i] = p.y ? p.write[i] : 0.f;
    rd[i] = p.read ? p.read[i] : 0.f;
  }
  if (p.y) {
#pragma unroll
    for (int i = 0; i < S * S; ++i) mix[i] = p.mix[i];
  }
  const T* yr = static_cast<const T*>(p.y) + (p.y ? row * p.ldy : 0);
  float ss = 0.f;
  for (int c = tid * V; c < W; c += 256 * V) {
    float x[S][V], y[V];
    if (p.embed) {
#pragma unroll
      for (int v = 0; v < V; ++v) {
        const float e = er ? ld(er + c + v) : 0.f;
#pragma unroll
        for (int s = 0; s < S; ++s) x[s][v] = e;
      }
    } else {
#pragma unroll
      for (int s = 0; s < S; ++s) {
        if constexpr (V == 4) {
          const f32x4_t t = ld4(xr + (int64_t)s * W + c);
#pragma unroll
          for (int v = 0; v < V; ++v) x[s][v] = t[v];
        } else {
          x[s][0] = xr[(int64_t)s * W + c];
        }
      }
    }
    if (p.y) {
#pragma unroll
      for (int v = 0; v < V; ++v) y[v] = p.bias ? p.bias[c + v] : 0.f;
      if constexpr (V == 4) {
        const f32x4_t t = ld4(yr + c);
#pragma unroll
        for (int v = 0; v < V; ++v) y[v] += t[v];
      } else {
        y[0] += ld(yr + c);
      }
      float n[S][V];
#pragma unroll
      for (int t = 0; t < S; ++t)
#pragma unroll
        for (int v = 0; v < V; ++v) {
          float a = wr[t] * y[v];
#pragma unroll
          for (int s = 0; s < S; ++s) a += mix[s * S + t] * x[s][v];
          n[t][v] = a;
        }
#pragma unroll
      for (int t = 0; t < S; ++t)
#pragma unroll
        for (int v = 0; v < V; ++v) x[t][v] = n[t][v];
    }
    if (p.store) {
#pragma unroll
      for (int s = 0; s < S; ++s) {
        if constexpr (V == 4)
          st4(xr + (int64_t)s * W + c, f32x4_t{x[s][0], x[s][1], x[s][2], x[s][3]});
        else
          xr[(int64_t)s * W + c] = x[s][0];
      }
    }
    if (p.read) {
#pragma unroll
      for (int v = 0; v < V; ++v) {
        float u = 0.f;
#pragma unroll
        for (int s = 0; s < S; ++s) u += rd[s] * x[s][v];
        us[c + v] = u;
        ss += u * u;
      }
    }
  }
  if (!p.read) return;
  const float rstd = 1.f / sqrtf(block_sum(ss, red) / (float)W + p.eps);
  T* hr = static_cast<T*>(p.h) + (int64_t)blockIdx.x * p.ldh;
  for (int c = tid * V; c < W; c += 256 * V) {   // a thread reads back only what it wrote
    if constexpr (V == 4) {
      const f32x4_t g = ld4(p.norm_w + c);
      const f32x4_t u = ld4(us + c);
      st4(hr + c, f32x4_t{u[0] * rstd * (1.f + g[0]), u[1] * rstd * (1.f + g[1]), u[2] * rstd * (1.f + g[2]),
                          u[3] * rstd * (1.f + g[3])});
    } else {
      st(hr + c, us[c] * rstd * (1.f + p.norm_w[c]));
    }
  }
}

// y = relu(x)^2
template <typename T>
__global__ void __launch_bounds__(256) relu_squared_kernel(const T* x, T* y, int64_t n) {
  for (int64_t i = ((int64_t)blockIdx.x * 256 + threadIdx.x) * 4; i < n; i += (int64_t)gridDim.x * 1024) {
    if (i + 4 <= n) {
      f32x4_t v = ld4(x + i);
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = v[j] > 0.f ? v[j] * v[j] : 0.f;
      st4(y + i, v);
    } else {
      for (int64_t j = i; j < n; ++j) {
        const float v = ld(x + j);
        st(y + j, v > 0.f ? v * v : 0.f);
      }
    }
  }
}

// x = cap * tanh(x / cap), in place (fp32)
__global__ void __launch_bounds__(256) softcap_kernel(float* x, int64_t n, float cap) {
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256)
    x[i] = cap * tanhf(x[i] / cap);
}

template <typename T, int S>
static int launch_hyper(const HyperParams& p, int64_t R, hipStream_t s) {
  const size_t lds = p.read ? (size_t)p.W * 4 : 0;
  if (p.W % 4 == 0 && p.ldy % 4 == 0 && p.ldh % 4 == 0)
    hipLaunchKernelGGL((hyper_step_kernel<T, S, 4>), dim3((unsigned)R), dim3(256), lds, s, p);
  else
    hipLaunchKernelGGL((hyper_step_kernel<T, S, 1>), dim3((unsigned)R), dim3(256), lds, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

template <typename T>
static int dispatch_hyper(const HyperParams& p, int S, int64_t R, hipStream_t s) {
  switch (S) {
    case 1: return launch_hyper<T, 1>(p, R, s);
    case 2: return launch_hyper<T, 2>(p, R, s);
    case 3: return launch_hyper<T, 3>(p, R, s);
    case 4: return launch_hyper<T, 4>(p, R, s);
    case 5: return launch_hyper<T, 5>(p, R, s);
    case 6: return launch_hyper<T, 6>(p, R, s);
    case 7: return launch_hyper<T, 7>(p, R, s);
    case 8: return launch_hyper<T, 8>(p, R, s);
  }
  return -1;
}

}  // namespace hybrid

int hyper_step_launch(bool f32, float* x, const void* embed, const int64_t* ids, int64_t vocab, const void* y, int64_t ldy,
                      const float* bias, const float* mix, const float* write, const float* read, const float* norm_w,
                      float eps, void* h, int64_t ldh, const int64_t* rows, bool store, int64_t R, int S, int W,
                      hipStream_t s) {
  if (R == 0) return 0;
  hybrid::HyperParams p{x, embed, ids, vocab, y, ldy, bias, mix, write, read, norm_w, eps, h, ldh, rows, store ? 1 : 0, W};
  return f32 ? hybrid::dispatch_hyper<float>(p, S, R, s) : hybrid::dispatch_hyper<uint16_t>(p, S, R, s);
}

int relu_squared_launch(bool f32, const void* x, void* y, int64_t n, hipStream_t s) {
  if (n == 0) return 0;
  const int64_t blocks = ceil_div64(n, 1024);
  const dim3 grid((unsigned)(blocks < 8192 ? blocks : 8192));
  if (f32)
    hipLaunchKernelGGL((hybrid::relu_squared_kernel<float>), grid, dim3(256), 0, s, static_cast<const float*>(x),
                       static_cast<float*>(y), n);
  else
    hipLaunchKernelGGL((hybrid::relu_squared_kernel<uint16_t>), grid, dim3(256), 0, s, static_cast<const uint16_t*>(x),
                       static_cast<uint16_t*>(y), n);
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

int softcap_launch(float* x, int64_t n, float cap, hipStream_t s) {
  if (n == 0) return 0;
  const int64_t blocks = ceil_div64(n, 256);
  hipLaunchKernelGGL(hybrid::softcap_kernel, dim3((unsigned)(blocks < 8192 ? blocks : 8192)), dim3(256), 0, s, x, n, cap);
  return hipGetLastError() == hipSuccess ? 0 : 1;
}

}  // namespace nxd
