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

}  // namespace

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
