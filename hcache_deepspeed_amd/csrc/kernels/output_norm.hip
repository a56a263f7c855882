// Norms on the output side of a sublayer, over a 32-bit residual stream:
//
//   x'  = x + g * norm(delta),   norm(d) = d / sqrt(mean(d^2) + eps)
//
// delta is a sublayer's output row, or the output of a routed expert layer that is summed here on the way in:
//
//   delta = sum_j w_j * (expert_j < E ? y[row_j] : x) + sigmoid(s) * shared
//
// (choices past the E experts are identities: they return their input). Also the embedding rows that start the stream,
// and the norm of the rows whose logits are asked for. Next to the 32-bit rows the kernels write the rows the next
// sublayer reads, rounded to the activations' type and zero-padded to a row length of the caller's choice.
//
// Layers with a norm on both sides of a sublayer run one kernel between two sublayers:
//
//   x'  = x + g * norm(delta),   y = gn * norm(x')
#include "hds_common.h"

namespace {
using namespace hds;

template <typename T>
struct ResidualNormParams {
  const float* x;  // [n, W]
  float* x_out;    // [n, W], may be x
  T* xb;           // [n, ldb] rounded rows or null
  int64_t ldb;
  const T* delta;  // [n, ldd]; null: the sum below
  int64_t ldd;
  const float* g;  // [W]; null: no norm and no residual, the sum itself goes to sum_out [n, W]
  T* sum_out;
  // expert sum
  const T* y;          // [rows, ldy]
  int64_t ldy;
  const int* expert;   // [n, k]
  const float* weight; // [n, k]
  const int* row;      // [n, k] row of y; null: n * k rows in order
  const T* shared;     // [n, lds] or null
  int64_t lds;
  const float* gate;   // [n] with stride ldg: s
  int64_t ldg;
  int E, k, identity;  // identity 0: the identity choices are left out (another rank adds them)
  int n, W;
  float eps;
};

template <typename T, int V>
__device__ __forceinline__ void load_delta(const ResidualNormParams<T>& p, int t, int c, float (&d)[V]) {
  if (p.delta != nullptr) {
    VecN<T, V>::load(p.delta + (int64_t)t * p.ldd + c, d);
    return;
  }
#pragma unroll
  for (int i = 0; i < V; ++i) d[i] = 0.f;
#pragma unroll 4
  for (int j = 0; j < p.k; ++j) {
    const int a = t * p.k + j, e = p.expert[a];
    float v[V];
    if (e < p.E) {
      VecN<T, V>::load(p.y + (int64_t)(p.row != nullptr ? max(p.row[a], 0) : a) * p.ldy + c, v);
    } else {
      if (!p.identity) continue;
      VecN<float, V>::load(p.x + (int64_t)t * p.W + c, v);
    }
    const float w = p.weight[a];
#pragma unroll
    for (int i = 0; i < V; ++i) d[i] += w * v[i];
  }
  if (p.shared != nullptr) {
    float v[V];
    VecN<T, V>::load(p.shared + (int64_t)t * p.lds + c, v);
    const float s = 1.f / (1.f + __expf(-p.gate[(int64_t)t * p.ldg]));
#pragma unroll
    for (int i = 0; i < V; ++i) d[i] += s * v[i];
  }
}

// one workgroup a row, the row (at most NC * V * 256 elements) in registers
template <typename T, int V, int NC>
__global__ __launch_bounds__(256) void residual_norm_kernel(ResidualNormParams<T> p) {
  __shared__ float red[4];
  constexpr int RT = 256;
  const int t = blockIdx.x, i0 = threadIdx.x;
  float d[NC][V], x[NC][V];
  float ss = 0.f;
#pragma unroll
  for (int q = 0; q < NC; ++q) {
    const int c = (i0 + q * RT) * V;
    if (c < p.W) {
      load_delta<T, V>(p, t, c, d[q]);
      if (p.g != nullptr) VecN<float, V>::load(p.x + (int64_t)t * p.W + c, x[q]);
#pragma unroll
      for (int i = 0; i < V; ++i) ss += d[q][i] * d[q][i];
    }
  }
  if (p.g == nullptr) {
#pragma unroll
    for (int q = 0; q < NC; ++q) {
      const int c = (i0 + q * RT) * V;
      if (c < p.W) VecN<T, V>::store(p.sum_out + (int64_t)t * p.W + c, d[q]);
    }
    return;
  }
  const float rs = 1.f / sqrtf(block_sum<256>(ss, red) / (float)p.W + p.eps);
#pragma unroll
  for (int q = 0; q < NC; ++q) {
    const int c = (i0 + q * RT) * V;
    if (c < p.W) {
      float g[V];
      VecN<float, V>::load(p.g + c, g);
#pragma unroll
      for (int i = 0; i < V; ++i) x[q][i] += d[q][i] * rs * g[i];
      VecN<float, V>::store(p.x_out + (int64_t)t * p.W + c, x[q]);
      if (p.xb != nullptr) VecN<T, V>::store(p.xb + (int64_t)t * p.ldb + c, x[q]);
    }
  }
  if (p.xb != nullptr)
    for (int c = p.W + i0; c < p.ldb; c += RT) p.xb[(int64_t)t * p.ldb + c] = from_f<T>(0.f);
}

// any width: the row's delta in LDS
template <typename T>
__global__ __launch_bounds__(256) void residual_norm_any_kernel(ResidualNormParams<T> p) {
  extern __shared__ float sm[];  // [4] reduction, [W] delta
  float* sd = sm + 4;
  const int t = blockIdx.x;
  float ss = 0.f;
  for (int c = threadIdx.x; c < p.W; c += 256) {
    float d[1];
    load_delta<T, 1>(p, t, c, d);
    sd[c] = d[0];
    ss += d[0] * d[0];
  }
  if (p.g == nullptr) {
    for (int c = threadIdx.x; c < p.W; c += 256) p.sum_out[(int64_t)t * p.W + c] = from_f<T>(sd[c]);
    return;
  }
  const float rs = 1.f / sqrtf(block_sum<256>(ss, sm) / (float)p.W + p.eps);
  for (int c = threadIdx.x; c < p.W; c += 256) {
    const float v = p.x[(int64_t)t * p.W + c] + sd[c] * rs * p.g[c];
    p.x_out[(int64_t)t * p.W + c] = v;
    if (p.xb != nullptr) p.xb[(int64_t)t * p.ldb + c] = from_f<T>(v);
  }
  if (p.xb != nullptr)
    for (int c = p.W + threadIdx.x; c < p.ldb; c += 256) p.xb[(int64_t)t * p.ldb + c] = from_f<T>(0.f);
}

template <typename T>
int launch_residual_norm(const ResidualNormParams<T>& p, hipStream_t st) {
  const bool v8 = p.W % 8 == 0 && p.ldb % 8 == 0 && p.ldd % 8 == 0 && p.ldy % 8 == 0 && p.lds % 8 == 0;
#define HDS_RN(NC) hipLaunchKernelGGL((residual_norm_kernel<T, 8, NC>), dim3(p.n), dim3(256), 0, st, p)
  if (v8 && p.W <= 16384) {
    if (p.W <= 2048) HDS_RN(1); else if (p.W <= 4096) HDS_RN(2); else if (p.W <= 8192) HDS_RN(4); else HDS_RN(8);
  } else {
    const size_t lds = (4 + (size_t)p.W) * sizeof(float);
    if (lds > 64 * 1024) return hipErrorInvalidValue;
    hipLaunchKernelGGL(residual_norm_any_kernel<T>, dim3(p.n), dim3(256), lds, st, p);
  }
#undef HDS_RN
  return hipGetLastError();
}

// x = embed[id] * scale, and its rounded copy
template <typename T, int V>
__global__ __launch_bounds__(256) void embed_rows_kernel(const T* __restrict__ embed, const int64_t* __restrict__ ids,
                                                         float scale, float* __restrict__ x, T* __restrict__ xb,
                                                         int64_t ldb, int W, int vocab) {
  const int64_t t = blockIdx.x;
  const int64_t id = min(max(ids[t], (int64_t)0), (int64_t)vocab - 1);
  for (int c = threadIdx.x * V; c < W; c += 256 * V) {
    float v[V];
    VecN<T, V>::load(embed + id * W + c, v);
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] *= scale;
    VecN<float, V>::store(x + t * W + c, v);
    if (xb != nullptr) VecN<T, V>::store(xb + t * ldb + c, v);
  }
  if (xb != nullptr)
    for (int c = W + threadIdx.x; c < ldb; c += 256) xb[t * ldb + c] = from_f<T>(0.f);
}

// y[i] = g * norm(x[idx[i]] + delta[idx[i]]): the output norm of the rows whose logits are asked for
template <typename T, int V>
__global__ __launch_bounds__(256) void norm_rows_kernel(const float* __restrict__ x, const T* __restrict__ delta,
                                                        const int* __restrict__ idx, const float* __restrict__ g,
                                                        int gs, T* __restrict__ y, int W, float eps) {
  __shared__ float red[4];
  const int64_t row = idx[blockIdx.x];
  auto load = [&](int c, float (&v)[V]) {
    VecN<float, V>::load(x + row * W + c, v);
    if (delta != nullptr) {
      float d[V];
      VecN<T, V>::load(delta + row * W + c, d);
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] += d[i];
    }
  };
  float ss = 0.f;
  for (int c = threadIdx.x * V; c < W; c += 256 * V) {
    float v[V];
    load(c, v);
#pragma unroll
    for (int i = 0; i < V; ++i) ss += v[i] * v[i];
  }
  const float rs = 1.f / sqrtf(block_sum<256>(ss, red) / (float)W + eps);
  for (int c = threadIdx.x * V; c < W; c += 256 * V) {
    float v[V];
    load(c, v);
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] = v[i] * rs * g[gs ? c + i : 0];
    VecN<T, V>::store(y + (int64_t)blockIdx.x * W + c, v);
  }
}

// ---------------------------------------------------------------------------------------------------------------
// norms on both sides
// ---------------------------------------------------------------------------------------------------------------
template <typename T>
struct SandwichParams {
  const float* x;      // [rows, W], or null: scale * embed[ids]
  const T* embed;
  const int64_t* ids;
  float scale;
  const T* delta;      // [rows, ldd] or null
  int64_t ldd;
  const float* g;      // [W]
  const float* gn;     // [W]
  const int* idx;      // [n] row of x and delta of every output row; null: 0 .. n - 1
  float* x_out;        // [n, W] or null; may be x when idx is null
  T* y;                // [n, W]
  int n, W, vocab;
  float eps;
};

template <typename T, int V>
__device__ __forceinline__ void load_x(const SandwichParams<T>& p, int64_t row, int64_t id, int c, float (&v)[V]) {
  if (p.x != nullptr) {
    VecN<float, V>::load(p.x + row * p.W + c, v);
  } else {
    VecN<T, V>::load(p.embed + id * p.W + c, v);
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] *= p.scale;
  }
}

// block-wide sum with one barrier; every call has its own `red`
template <int NT>
__device__ __forceinline__ float block_sum_once(float v, float* red) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float r = 0.f;
#pragma unroll
  for (int i = 0; i < NT / 64; ++i) r += red[i];
  return r;
}

// one workgroup a row; the row (at most NC * V * NT elements) and all it needs in registers
template <typename T, int V, int NC, int NT>
__global__ __launch_bounds__(NT) void sandwich_norm_kernel(SandwichParams<T> p) {
  __shared__ float red[2][NT / 64];
  const int64_t t = blockIdx.x, row = p.idx != nullptr ? p.idx[t] : t;
  const int64_t id = p.x == nullptr ? min(max(p.ids[row], (int64_t)0), (int64_t)p.vocab - 1) : 0;
  float x[NC][V], d[NC][V], g[NC][V], gn[NC][V];
  float ss = 0.f;
#pragma unroll
  for (int q = 0; q < NC; ++q) {
    const int c = (q * NT + threadIdx.x) * V;
    if (c < p.W) {
      load_x<T, V>(p, row, id, c, x[q]);
      VecN<float, V>::load(p.gn + c, gn[q]);
      if (p.delta != nullptr) {
        VecN<T, V>::load(p.delta + row * p.ldd + c, d[q]);
        VecN<float, V>::load(p.g + c, g[q]);
#pragma unroll
        for (int i = 0; i < V; ++i) ss += d[q][i] * d[q][i];
      }
    }
  }
  const float rd = p.delta != nullptr ? 1.f / sqrtf(block_sum_once<NT>(ss, red[0]) / (float)p.W + p.eps) : 0.f;
  ss = 0.f;
#pragma unroll
  for (int q = 0; q < NC; ++q) {
    const int c = (q * NT + threadIdx.x) * V;
    if (c < p.W) {
#pragma unroll
      for (int i = 0; i < V; ++i) {
        if (p.delta != nullptr) x[q][i] += d[q][i] * rd * g[q][i];
        ss += x[q][i] * x[q][i];
      }
      if (p.x_out != nullptr) VecN<float, V>::store(p.x_out + t * p.W + c, x[q]);
    }
  }
  const float rx = 1.f / sqrtf(block_sum_once<NT>(ss, red[1]) / (float)p.W + p.eps);
#pragma unroll
  for (int q = 0; q < NC; ++q) {
    const int c = (q * NT + threadIdx.x) * V;
    if (c < p.W) {
#pragma unroll
      for (int i = 0; i < V; ++i) x[q][i] *= rx * gn[q][i];
      VecN<T, V>::store(p.y + t * p.W + c, x[q]);
    }
  }
}

// any width: the row in LDS
template <typename T>
__global__ __launch_bounds__(256) void sandwich_norm_any_kernel(SandwichParams<T> p) {
  extern __shared__ float sm[];  // [2][4] reductions, [W] row
  float* sx = sm + 8;
  const int64_t t = blockIdx.x, row = p.idx != nullptr ? p.idx[t] : t;
  const int64_t id = p.x == nullptr ? min(max(p.ids[row], (int64_t)0), (int64_t)p.vocab - 1) : 0;
  float ss = 0.f;
  if (p.delta != nullptr)
    for (int c = threadIdx.x; c < p.W; c += 256) {
      const float d = to_f(p.delta[row * p.ldd + c]);
      ss += d * d;
    }
  const float rd = 1.f / sqrtf(block_sum_once<256>(ss, sm) / (float)p.W + p.eps);
  ss = 0.f;
  for (int c = threadIdx.x; c < p.W; c += 256) {
    float v[1];
    load_x<T, 1>(p, row, id, c, v);
    if (p.delta != nullptr) v[0] += to_f(p.delta[row * p.ldd + c]) * rd * p.g[c];
    sx[c] = v[0];
    ss += v[0] * v[0];
    if (p.x_out != nullptr) p.x_out[t * p.W + c] = v[0];
  }
  const float rx = 1.f / sqrtf(block_sum_once<256>(ss, sm + 4) / (float)p.W + p.eps);
  for (int c = threadIdx.x; c < p.W; c += 256) p.y[t * p.W + c] = from_f<T>(sx[c] * rx * p.gn[c]);
}

template <typename T>
int launch_sandwich(const SandwichParams<T>& p, hipStream_t st) {
#define HDS_SN(V, NC, NT) hipLaunchKernelGGL((sandwich_norm_kernel<T, V, NC, NT>), dim3(p.n), dim3(NT), 0, st, p)
  if (p.n <= 64 && p.W % 4 == 0 && p.ldd % 4 == 0 && p.W <= 8192) {  // few rows: many threads on each
    if (p.W <= 1024) HDS_SN(4, 1, 256); else if (p.W <= 4096) HDS_SN(4, 1, 1024); else HDS_SN(4, 2, 1024);
  } else if (p.W % 8 == 0 && p.ldd % 8 == 0 && p.W <= 8192) {
    if (p.W <= 2048) HDS_SN(8, 1, 256); else if (p.W <= 4096) HDS_SN(8, 1, 512); else HDS_SN(8, 1, 1024);
  } else {
    const size_t lds = (8 + (size_t)p.W) * sizeof(float);
    if (lds > 64 * 1024) return hipErrorInvalidValue;
    hipLaunchKernelGGL(sandwich_norm_any_kernel<T>, dim3(p.n), dim3(256), lds, st, p);
  }
#undef HDS_SN
  return hipGetLastError();
}

// y = w * norm(x) of [n, W] rows with row stride ld: one wave a row
template <typename T, int V>
__global__ __launch_bounds__(256) void row_norm_kernel(const T* __restrict__ x, int64_t ld, const float* __restrict__ w,
                                                       T* __restrict__ y, int64_t ldy, int n, int W, float eps) {
  const int64_t t = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (t >= n) return;
  const int lane = threadIdx.x & 63;
  constexpr int KEEP = 32 / V;  // chunks kept in registers (rows up to 2048)
  float v[KEEP][V], ss = 0.f;
#pragma unroll
  for (int q = 0; q < KEEP; ++q) {
    const int c = (q * 64 + lane) * V;
    if (c < W) {
      VecN<T, V>::load(x + t * ld + c, v[q]);
#pragma unroll
      for (int i = 0; i < V; ++i) ss += v[q][i] * v[q][i];
    }
  }
  for (int c = (KEEP * 64 + lane) * V; c < W; c += 64 * V) {
    float u[V];
    VecN<T, V>::load(x + t * ld + c, u);
#pragma unroll
    for (int i = 0; i < V; ++i) ss += u[i] * u[i];
  }
  const float rs = 1.f / sqrtf(wave_sum(ss) / (float)W + eps);
#pragma unroll
  for (int q = 0; q < KEEP; ++q) {
    const int c = (q * 64 + lane) * V;
    if (c < W) {
      float g[V];
      VecN<float, V>::load(w + c, g);
#pragma unroll
      for (int i = 0; i < V; ++i) v[q][i] *= rs * g[i];
      VecN<T, V>::store(y + t * ldy + c, v[q]);
    }
  }
  for (int c = (KEEP * 64 + lane) * V; c < W; c += 64 * V) {
    float u[V], g[V];
    VecN<T, V>::load(x + t * ld + c, u);
    VecN<float, V>::load(w + c, g);
#pragma unroll
    for (int i = 0; i < V; ++i) u[i] *= rs * g[i];
    VecN<T, V>::store(y + t * ldy + c, u);
  }
}

// x = cap * tanh(x / cap)
template <typename T>
__global__ __launch_bounds__(256) void softcap_kernel(T* __restrict__ x, int64_t n, float cap) {
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256)
    x[i] = from_f<T>(cap * tanhf(to_f(x[i]) / cap));
}

}  // namespace

// x' = x + g * norm(delta) to x_out (null: not kept) and gn * norm(x') to y, of rows idx (null: all n). x null: the
// stream starts with the rows scale * embed[ids]; delta null: x' = x.
HDS_EXPORT int hds_sandwich_norm(int dtype, const float* x, const void* embed, const int64_t* ids, float scale,
                                 const void* delta, int64_t ldd, const float* g, const float* gn, const int* idx,
                                 float* x_out, void* y, int n, int W, int vocab, float eps, hipStream_t st) {
  if (n <= 0) return 0;
  if (W < 1 || gn == nullptr || y == nullptr || (x == nullptr && (embed == nullptr || ids == nullptr || vocab < 1)) ||
      (delta != nullptr && (g == nullptr || ldd < W)) || (idx != nullptr && x_out != nullptr && x_out == x))
    return hipErrorInvalidValue;
#define HDS_SW(TT)                                                                                              \
  return launch_sandwich(SandwichParams<TT>{x, (const TT*)embed, ids, scale, (const TT*)delta, ldd, g, gn, idx, \
                                            x_out, (TT*)y, n, W, vocab, eps}, st)
  if (dtype == kBF16) HDS_SW(bf16);
  if (dtype == kF32) HDS_SW(float);
#undef HDS_SW
  return hipErrorInvalidValue;
}

HDS_EXPORT int hds_row_norm(int dtype, const void* x, int64_t ld, const float* w, void* y, int64_t ldy, int n, int W,
                            float eps, hipStream_t st) {
  if (n <= 0) return 0;
  if (W < 1 || ld < W || ldy < W || w == nullptr) return hipErrorInvalidValue;
  const bool v8 = W % 8 == 0 && ld % 8 == 0 && ldy % 8 == 0 && (uintptr_t)x % 16 == 0 && (uintptr_t)y % 16 == 0;
#define HDS_RW(TT, VV)                                                                                            \
  hipLaunchKernelGGL((row_norm_kernel<TT, VV>), dim3((n + 3) / 4), dim3(256), 0, st, (const TT*)x, ld, w, (TT*)y, \
                     ldy, n, W, eps)
  if (dtype == kBF16) {
    if (v8) HDS_RW(bf16, 8); else HDS_RW(bf16, 1);
  } else if (dtype == kF32) {
    if (v8) HDS_RW(float, 8); else HDS_RW(float, 1);
  } else {
    return hipErrorInvalidValue;
  }
#undef HDS_RW
  return hipGetLastError();
}

// n contiguous values in place
HDS_EXPORT int hds_softcap(int dtype, void* x, int64_t n, float cap, hipStream_t st) {
  if (n <= 0) return 0;
  if (!(cap > 0.f)) return hipErrorInvalidValue;
  const dim3 grid(stream_grid(n, 256));
  if (dtype == kBF16) hipLaunchKernelGGL(softcap_kernel<bf16>, grid, dim3(256), 0, st, (bf16*)x, n, cap);
  else if (dtype == kF32) hipLaunchKernelGGL(softcap_kernel<float>, grid, dim3(256), 0, st, (float*)x, n, cap);
  else return hipErrorInvalidValue;
  return hipGetLastError();
}

// One sublayer output row per residual row; x_out may be x.
HDS_EXPORT int hds_residual_norm(int dtype, const float* x, float* x_out, void* xb, int64_t ldb, const void* delta,
                                 int64_t ldd, const float* g, int n, int W, float eps, hipStream_t st) {
  if (n <= 0) return 0;
  if (W < 1 || delta == nullptr || g == nullptr || ldd < W || (xb != nullptr && ldb < W)) return hipErrorInvalidValue;
#define HDS_RN(TT)                                                                                                 \
  return launch_residual_norm(ResidualNormParams<TT>{x, x_out, (TT*)xb, ldb, (const TT*)delta, ldd, g, nullptr,   \
                                                     nullptr, 0, nullptr, nullptr, nullptr, nullptr, 0, nullptr,  \
                                                     0, 0, 0, 0, n, W, eps}, st)
  if (dtype == kBF16) HDS_RN(bf16);
  if (dtype == kF32) HDS_RN(float);
#undef HDS_RN
  return hipErrorInvalidValue;
}

// The expert sum of every row, then the residual norm; g null: the sum goes to sum_out instead (x is read for the
// identity choices only).
HDS_EXPORT int hds_experts_norm(int dtype, const float* x, float* x_out, void* xb, int64_t ldb, const float* g,
                                void* sum_out, const void* y, int64_t ldy, const int* expert, const float* weight,
                                const int* row, const void* shared, int64_t lds, const float* gate, int64_t ldg, int E,
                                int k, int identity, int n, int W, float eps, hipStream_t st) {
  if (n <= 0) return 0;
  if (W < 1 || k < 1 || E < 1 || y == nullptr || ldy < W || expert == nullptr || weight == nullptr || x == nullptr ||
      (shared != nullptr && (lds < W || gate == nullptr)) || (g == nullptr ? sum_out == nullptr : x_out == nullptr) ||
      (xb != nullptr && ldb < W))
    return hipErrorInvalidValue;
#define HDS_RN(TT)                                                                                                  \
  return launch_residual_norm(ResidualNormParams<TT>{x, x_out, (TT*)xb, ldb, nullptr, 0, g, (TT*)sum_out,          \
                                                     (const TT*)y, ldy, expert, weight, row, (const TT*)shared,    \
                                                     lds, gate, ldg, E, k, identity, n, W, eps}, st)
  if (dtype == kBF16) HDS_RN(bf16);
  if (dtype == kF32) HDS_RN(float);
#undef HDS_RN
  return hipErrorInvalidValue;
}

HDS_EXPORT int hds_embed_rows(int dtype, const void* embed, const int64_t* ids, float scale, float* x, void* xb,
                              int64_t ldb, int n, int W, int vocab, hipStream_t st) {
  if (n <= 0) return 0;
  if (W < 1 || vocab < 1 || (xb != nullptr && ldb < W)) return hipErrorInvalidValue;
  const bool v8 = W % 8 == 0 && ldb % 8 == 0;
#define HDS_ER(TT, VV)                                                                                             \
  hipLaunchKernelGGL((embed_rows_kernel<TT, VV>), dim3(n), dim3(256), 0, st, (const TT*)embed, ids, scale, x,     \
                     (TT*)xb, ldb, W, vocab)
  if (dtype == kBF16) {
    if (v8) HDS_ER(bf16, 8); else HDS_ER(bf16, 1);
  } else if (dtype == kF32) {
    if (v8) HDS_ER(float, 8); else HDS_ER(float, 1);
  } else {
    return hipErrorInvalidValue;
  }
#undef HDS_ER
  return hipGetLastError();
}

// delta may be null
HDS_EXPORT int hds_norm_rows(int dtype, const float* x, const void* delta, const int* idx, const float* g, int gs,
                             void* y, int n_rows, int W, float eps, hipStream_t st) {
  if (n_rows <= 0) return 0;
  const bool v4 = W % 4 == 0;
#define HDS_NR(TT, VV)                                                                                             \
  hipLaunchKernelGGL((norm_rows_kernel<TT, VV>), dim3(n_rows), dim3(256), 0, st, x, (const TT*)delta, idx, g, gs, \
                     (TT*)y, W, eps)
  if (dtype == kBF16) {
    if (v4) HDS_NR(bf16, 4); else HDS_NR(bf16, 1);
  } else if (dtype == kF32) {
    if (v4) HDS_NR(float, 4); else HDS_NR(float, 1);
  } else {
    return hipErrorInvalidValue;
  }
#undef HDS_NR
  return hipGetLastError();
}
