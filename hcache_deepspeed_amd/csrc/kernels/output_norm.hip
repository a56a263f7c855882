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
//   x'  = x + N(delta),   y = N'(x')
//
// where N and N' are RMS norms with a gain or layer norms with a gain and a bias (norm(d) = (d - mean) / sqrt(mean((d -
// mean)^2) + eps)), N' may be absent (y is x', rounded), and delta is a sublayer's output, an expert sum as above, or half the
// sum of two outputs that are RMS-normed first:
//
//   delta = (ga * rms(a) + gb * rms(b)) / 2
#include "hds_common.h"

namespace {
using namespace hds;

// sum over the chosen experts
template <typename T>
struct ExpertParts {
  const T* y;          // [rows, ldy]
  int64_t ldy;
  const int* expert;   // [n, k]
  const float* weight; // [n, k] or null: ones
  const int* row;      // [n, k] row of y; null: n * k rows in order
  const T* shared;     // [n, lds] or null
  int64_t lds;
  const float* gate;   // [n] with stride ldg: s
  int64_t ldg;
  int E, k, identity;  // identity 0: the identity choices are left out (another rank adds them)
};

// V columns from c of row t; x: the row's residual
template <typename T, int V>
__device__ __forceinline__ void load_parts(const ExpertParts<T>& p, const float* x, int64_t t, int c, float (&d)[V]) {
#pragma unroll
  for (int i = 0; i < V; ++i) d[i] = 0.f;
#pragma unroll 4
  for (int j = 0; j < p.k; ++j) {
    const int64_t a = t * p.k + j;
    const int e = p.expert[a];
    float v[V];
    if (e < p.E) {
      VecN<T, V>::load(p.y + (p.row != nullptr ? max(p.row[a], 0) : a) * p.ldy + c, v);
    } else {
      if (!p.identity) continue;
      VecN<float, V>::load(x + c, v);
    }
    const float w = p.weight != nullptr ? p.weight[a] : 1.f;
#pragma unroll
    for (int i = 0; i < V; ++i) d[i] += w * v[i];
  }
  if (p.shared != nullptr) {
    float v[V];
    VecN<T, V>::load(p.shared + t * p.lds + c, v);
    const float s = 1.f / (1.f + __expf(-p.gate[t * p.ldg]));
#pragma unroll
    for (int i = 0; i < V; ++i) d[i] += s * v[i];
  }
}

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
  ExpertParts<T> parts;
  int n, W;
  float eps;
};

template <typename T, int V>
__device__ __forceinline__ void load_delta(const ResidualNormParams<T>& p, int t, int c, float (&d)[V]) {
  if (p.delta != nullptr) {
    VecN<T, V>::load(p.delta + (int64_t)t * p.ldd + c, d);
    return;
  }
  load_parts<T, V>(p.parts, p.x + (int64_t)t * p.W, t, c, d);
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
  const bool v8 = p.W % 8 == 0 && p.ldb % 8 == 0 && p.ldd % 8 == 0 && p.parts.ldy % 8 == 0 && p.parts.lds % 8 == 0;
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

// The general step: layer norms, a pair or an expert sum as delta, no second norm, padded rows
enum Delta : int { kPlain = 0, kPair = 1, kExperts = 2 };

template <typename T>
struct StreamParams {
  const float* x;       // [rows, W]
  const T* delta;       // [rows, ldd] or null (kPlain)
  int64_t ldd;
  const T* other;       // kPair: [rows, ldo]
  int64_t ldo;
  const float* ga;      // kPair: [W]
  const float* gb;
  ExpertParts<T> parts; // kExperts
  const float* g;       // [W] gain of N
  const float* b;       // [W] bias: N is a layer norm; null: an RMS norm
  const float* gn;      // [W] gain of N'; null: none
  const float* bn;      // [W] or null, as b
  const int* idx;       // [n] row of every output row; null: 0 .. n - 1
  float* x_out;         // [n, W] or null; may be x when idx is null
  T* y;                 // [n, ldy] zero-filled behind W, or null
  int64_t ldy;
  int n, W;
  float eps;
};

// sums of two values in every thread with one barrier; every call has its own `red`
template <int NT>
__device__ __forceinline__ void block_sums(float& a, float& b, float* red) {
  a = wave_sum(a);
  b = wave_sum(b);
  if ((threadIdx.x & 63) == 0) {
    red[threadIdx.x >> 6] = a;
    red[NT / 64 + (threadIdx.x >> 6)] = b;
  }
  __syncthreads();
  a = b = 0.f;
#pragma unroll
  for (int i = 0; i < NT / 64; ++i) {
    a += red[i];
    b += red[NT / 64 + i];
  }
}

// Mean (0 for an RMS norm) and factor of a row whose elements every(f) passes to f
template <int NT, typename Every>
__device__ __forceinline__ void norm_of(bool layer, int W, float eps, float* red, Every&& every, float& mean, float& rs) {
  mean = 0.f;
  if (layer) {
    float sum = 0.f;
    every([&](float v) { sum += v; });
    mean = block_sum_once<NT>(sum, red) / (float)W;
  }
  float ss = 0.f;
  every([&](float v) { ss += (v - mean) * (v - mean); });
  rs = 1.f / sqrtf(block_sum_once<NT>(ss, red + NT / 64) / (float)W + eps);
}

// one workgroup a row, the row (at most NC * V * NT elements) in registers
template <typename T, int V, int NC, int NT, int D>
__global__ __launch_bounds__(NT) void stream_norm_kernel(StreamParams<T> p) {
  __shared__ float red[6 * (NT / 64)];
  const int64_t t = blockIdx.x, row = p.idx != nullptr ? p.idx[t] : t;
  float x[NC][V], d[NC][V];
  auto columns = [&](auto&& f) {
#pragma unroll
    for (int q = 0; q < NC; ++q) {
      const int c = (q * NT + threadIdx.x) * V;
      if (c < p.W) f(q, c);
    }
  };
  auto of = [&](float (&a)[NC][V]) {
    return [&](auto&& f) {
      columns([&](int q, int) {
#pragma unroll
        for (int i = 0; i < V; ++i) f(a[q][i]);
      });
    };
  };
  columns([&](int q, int c) { VecN<float, V>::load(p.x + row * p.W + c, x[q]); });
  bool adds = true;
  if constexpr (D == kPlain) {
    adds = p.delta != nullptr;
    if (adds) columns([&](int q, int c) { VecN<T, V>::load(p.delta + row * p.ldd + c, d[q]); });
  } else if constexpr (D == kExperts) {
    columns([&](int q, int c) { load_parts<T, V>(p.parts, p.x + row * p.W, row, c, d[q]); });
  } else {
    float o[NC][V], sa = 0.f, sb = 0.f;
    columns([&](int q, int c) {
      VecN<T, V>::load(p.delta + row * p.ldd + c, d[q]);
      VecN<T, V>::load(p.other + row * p.ldo + c, o[q]);
#pragma unroll
      for (int i = 0; i < V; ++i) {
        sa += d[q][i] * d[q][i];
        sb += o[q][i] * o[q][i];
      }
    });
    block_sums<NT>(sa, sb, red);
    const float ra = 0.5f / sqrtf(sa / (float)p.W + p.eps), rb = 0.5f / sqrtf(sb / (float)p.W + p.eps);
    columns([&](int q, int c) {
      float ga[V], gb[V];
      VecN<float, V>::load(p.ga + c, ga);
      VecN<float, V>::load(p.gb + c, gb);
#pragma unroll
      for (int i = 0; i < V; ++i) d[q][i] = d[q][i] * ra * ga[i] + o[q][i] * rb * gb[i];
    });
  }
  float mean, rs;
  if (adds) {
    norm_of<NT>(p.b != nullptr, p.W, p.eps, red + 2 * (NT / 64), of(d), mean, rs);
    columns([&](int q, int c) {
      float g[V];
      VecN<float, V>::load(p.g + c, g);
#pragma unroll
      for (int i = 0; i < V; ++i) x[q][i] += (d[q][i] - mean) * rs * g[i];
      if (p.b != nullptr) {
        VecN<float, V>::load(p.b + c, g);
#pragma unroll
        for (int i = 0; i < V; ++i) x[q][i] += g[i];
      }
    });
  }
  if (p.x_out != nullptr) columns([&](int q, int c) { VecN<float, V>::store(p.x_out + t * p.W + c, x[q]); });
  if (p.y == nullptr) return;
  if (p.gn != nullptr) {
    norm_of<NT>(p.bn != nullptr, p.W, p.eps, red + 4 * (NT / 64), of(x), mean, rs);
    columns([&](int q, int c) {
      float g[V], b[V];
      VecN<float, V>::load(p.gn + c, g);
#pragma unroll
      for (int i = 0; i < V; ++i) b[i] = 0.f;
      if (p.bn != nullptr) VecN<float, V>::load(p.bn + c, b);
#pragma unroll
      for (int i = 0; i < V; ++i) x[q][i] = (x[q][i] - mean) * rs * g[i] + b[i];
    });
  }
  columns([&](int q, int c) { VecN<T, V>::store(p.y + t * p.ldy + c, x[q]); });
  for (int c = p.W + threadIdx.x; c < p.ldy; c += NT) p.y[t * p.ldy + c] = from_f<T>(0.f);
}

// any width: the row in LDS
template <typename T, int D>
__global__ __launch_bounds__(256) void stream_norm_any_kernel(StreamParams<T> p) {
  extern __shared__ float sm[];  // [6][4] reductions, [W] row
  float* sx = sm + 24;
  const int64_t t = blockIdx.x, row = p.idx != nullptr ? p.idx[t] : t;
  auto every = [&](auto&& f) {
    for (int c = threadIdx.x; c < p.W; c += 256) f(sx[c]);
  };
  const float* x = p.x + row * p.W;
  bool adds = true;
  if constexpr (D == kPlain) {
    adds = p.delta != nullptr;
    if (adds)
      for (int c = threadIdx.x; c < p.W; c += 256) sx[c] = to_f(p.delta[row * p.ldd + c]);
  } else if constexpr (D == kExperts) {
    for (int c = threadIdx.x; c < p.W; c += 256) {
      float v[1];
      load_parts<T, 1>(p.parts, x, row, c, v);
      sx[c] = v[0];
    }
  } else {
    float sa = 0.f, sb = 0.f;
    for (int c = threadIdx.x; c < p.W; c += 256) {
      const float a = to_f(p.delta[row * p.ldd + c]), b = to_f(p.other[row * p.ldo + c]);
      sa += a * a;
      sb += b * b;
    }
    block_sums<256>(sa, sb, sm);
    const float ra = 0.5f / sqrtf(sa / (float)p.W + p.eps), rb = 0.5f / sqrtf(sb / (float)p.W + p.eps);
    for (int c = threadIdx.x; c < p.W; c += 256)
      sx[c] = to_f(p.delta[row * p.ldd + c]) * ra * p.ga[c] + to_f(p.other[row * p.ldo + c]) * rb * p.gb[c];
  }
  // (a thread only reads the elements it wrote)
  float mean = 0.f, rs = 0.f;
  if (adds) norm_of<256>(p.b != nullptr, p.W, p.eps, sm + 8, every, mean, rs);
  for (int c = threadIdx.x; c < p.W; c += 256) {
    float v = x[c];
    if (adds) v += (sx[c] - mean) * rs * p.g[c] + (p.b != nullptr ? p.b[c] : 0.f);
    sx[c] = v;
    if (p.x_out != nullptr) p.x_out[t * p.W + c] = v;
  }
  if (p.y == nullptr) return;
  if (p.gn != nullptr) norm_of<256>(p.bn != nullptr, p.W, p.eps, sm + 16, every, mean, rs);
  for (int c = threadIdx.x; c < p.W; c += 256)
    p.y[t * p.ldy + c] = from_f<T>(p.gn == nullptr ? sx[c] : (sx[c] - mean) * rs * p.gn[c] + (p.bn != nullptr ? p.bn[c] : 0.f));
  for (int c = p.W + threadIdx.x; c < p.ldy; c += 256) p.y[t * p.ldy + c] = from_f<T>(0.f);
}

template <typename T, int D>
int launch_stream(const StreamParams<T>& p, hipStream_t st) {
#define HDS_ST(V, NC, NT) hipLaunchKernelGGL((stream_norm_kernel<T, V, NC, NT, D>), dim3(p.n), dim3(NT), 0, st, p)
  const int64_t lds_any = p.ldd | p.ldo | p.parts.ldy | p.parts.lds | p.ldy;
  if (p.n <= 64 && p.W % 4 == 0 && lds_any % 4 == 0 && p.W <= 8192) {  // few rows: many threads on each
    if (p.W <= 1024) HDS_ST(4, 1, 256); else if (p.W <= 4096) HDS_ST(4, 1, 1024); else HDS_ST(4, 2, 1024);
  } else if (p.W % 8 == 0 && lds_any % 8 == 0 && p.W <= 8192) {
    if (p.W <= 2048) HDS_ST(8, 1, 256); else if (p.W <= 4096) HDS_ST(8, 1, 512); else HDS_ST(8, 1, 1024);
  } else {
    const size_t lds = (24 + (size_t)p.W) * sizeof(float);
    if (lds > 64 * 1024) return hipErrorInvalidValue;
    hipLaunchKernelGGL((stream_norm_any_kernel<T, D>), dim3(p.n), dim3(256), lds, st, p);
  }
#undef HDS_ST
  return hipGetLastError();
}

// x = scale * embed[id] + pairs[(previous id * mul_prev + id * mul_cur) mod buckets], the last row of `pairs` for a sequence's
// first token. The previous token of a portion's first one is in the sequence's slot (its bits in a float's place).
template <typename T, int V>
__global__ __launch_bounds__(256) void embed_pairs_kernel(const T* __restrict__ embed, const T* __restrict__ pairs,
                                                          const int64_t* __restrict__ ids, float scale,
                                                          const int* __restrict__ tok_seq, const int* __restrict__ seq_meta,
                                                          const int* __restrict__ slots, int* state, int64_t slot_stride,
                                                          float* __restrict__ x, int W, int vocab, int buckets,
                                                          int64_t mul_prev, int64_t mul_cur) {
  __shared__ int s_prev;
  const int64_t t = blockIdx.x;
  const int s = tok_seq[t], q0 = seq_meta[3 * s], n = seq_meta[3 * s + 1], seen = seq_meta[3 * s + 2];
  auto valid = [&](int64_t id) { return min(max(id, (int64_t)0), (int64_t)vocab - 1); };
  const int64_t id = valid(ids[t]);
  if (threadIdx.x == 0) {
    if (t > q0) {
      s_prev = (int)valid(ids[t - 1]);
    } else {  // reads what earlier steps left, then leaves this step's last token
      int* at = state + (int64_t)slots[s] * slot_stride;
      s_prev = seen > 0 ? (int)valid(*at) : -1;
      *at = (int)valid(ids[q0 + n - 1]);
    }
  }
  __syncthreads();
  const int64_t prev = s_prev;
  const int64_t at = prev < 0 ? buckets : (prev * mul_prev + id * mul_cur) % buckets;
  for (int c = threadIdx.x * V; c < W; c += 256 * V) {
    float v[V], u[V];
    VecN<T, V>::load(embed + id * W + c, v);
    VecN<T, V>::load(pairs + at * W + c, u);
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] = v[i] * scale + u[i];
    VecN<float, V>::store(x + t * W + c, v);
  }
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
                                                     ExpertParts<TT>{}, n, W, eps}, st)
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
  if (W < 1 || k < 1 || E < 1 || y == nullptr || ldy < W || expert == nullptr || x == nullptr ||
      (shared != nullptr && (lds < W || gate == nullptr)) || (g == nullptr ? sum_out == nullptr : x_out == nullptr) ||
      (xb != nullptr && ldb < W))
    return hipErrorInvalidValue;
#define HDS_RN(TT)                                                                                                  \
  return launch_residual_norm(                                                                                      \
      ResidualNormParams<TT>{x, x_out, (TT*)xb, ldb, nullptr, 0, g, (TT*)sum_out,                                   \
                             ExpertParts<TT>{(const TT*)y, ldy, expert, weight, row, (const TT*)shared, lds, gate, \
                                             ldg, E, k, identity}, n, W, eps}, st)
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

// The general step between two sublayers (see StreamParams). kind: 0 delta is a matrix or null, 1 a pair, 2 an expert sum.
HDS_EXPORT int hds_stream_norm(int dtype, int kind, const float* x, const void* delta, int64_t ldd, const void* other,
                               int64_t ldo, const float* ga, const float* gb, const void* py, int64_t ldpy,
                               const int* expert, const float* weight, const int* prow, const void* shared, int64_t lds,
                               const float* gate, int64_t ldg, int E, int k, int identity, const float* g, const float* b,
                               const float* gn, const float* bn, const int* idx, float* x_out, void* y, int64_t ldy, int n,
                               int W, float eps, hipStream_t st) {
  if (n <= 0) return 0;
  if (W < 1 || x == nullptr || kind < 0 || kind > 2 || (y != nullptr && ldy < W) || (x_out == nullptr && y == nullptr) ||
      (idx != nullptr && x_out != nullptr && x_out == x) || ((kind > 0 || delta != nullptr) && g == nullptr) ||
      (kind < 2 && delta != nullptr && ldd < W) || (gn == nullptr && bn != nullptr))
    return hipErrorInvalidValue;
  if (kind == kPair && (delta == nullptr || other == nullptr || ldo < W || ga == nullptr || gb == nullptr))
    return hipErrorInvalidValue;
  if (kind == kExperts && (py == nullptr || ldpy < W || expert == nullptr || E < 1 || k < 1 ||
                           (shared != nullptr && (lds < W || gate == nullptr))))
    return hipErrorInvalidValue;
#define HDS_SX(TT)                                                                                                       \
  {                                                                                                                      \
    const StreamParams<TT> p{x, (const TT*)delta, ldd, (const TT*)other, ldo, ga, gb,                                   \
                             ExpertParts<TT>{(const TT*)py, ldpy, expert, weight, prow, (const TT*)shared, lds, gate,   \
                                             ldg, E, k, identity}, g, b, gn, bn, idx, x_out, (TT*)y, ldy, n, W, eps};   \
    return kind == kPlain ? launch_stream<TT, kPlain>(p, st)                                                             \
                          : kind == kPair ? launch_stream<TT, kPair>(p, st) : launch_stream<TT, kExperts>(p, st);        \
  }
  if (dtype == kBF16) HDS_SX(bf16)
  if (dtype == kF32) HDS_SX(float)
#undef HDS_SX
  return hipErrorInvalidValue;
}

// pairs [buckets + 1, W]; state: the place of the last token in the first slot; slot_stride in 4-byte units
HDS_EXPORT int hds_embed_pairs(int dtype, const void* embed, const void* pairs, const int64_t* ids, float scale,
                               const int* tok_seq, const int* seq_meta, const int* slots, void* state,
                               int64_t slot_stride, float* x, int n, int W, int vocab, int buckets, int64_t mul_prev,
                               int64_t mul_cur, hipStream_t st) {
  if (n <= 0) return 0;
  if (W < 1 || vocab < 1 || buckets < 1 || mul_prev < 0 || mul_cur < 0 || state == nullptr || slot_stride < 1)
    return hipErrorInvalidValue;
#define HDS_EP(TT, VV)                                                                                                  \
  hipLaunchKernelGGL((embed_pairs_kernel<TT, VV>), dim3(n), dim3(256), 0, st, (const TT*)embed, (const TT*)pairs, ids, \
                     scale, tok_seq, seq_meta, slots, (int*)state, slot_stride, x, W, vocab, buckets, mul_prev, mul_cur)
  if (dtype == kBF16) {
    if (W % 8 == 0) HDS_EP(bf16, 8); else HDS_EP(bf16, 1);
  } else if (dtype == kF32) {
    if (W % 8 == 0) HDS_EP(float, 8); else HDS_EP(float, 1);
  } else {
    return hipErrorInvalidValue;
  }
#undef HDS_EP
  return hipGetLastError();
}
