// Pre-norm of a serving layer with a 32-bit residual stream and a causal input convolution, in one launch:
//
//   x'   = x + delta                       (32-bit residual; x may also be the embedding rows of the step's tokens)
//   u    = x' / sqrt(mean(x'^2) + eps)
//   h_k  = g_k * u                         (k = 0, 1: a layer's two sublayers may read the same normed row; g_k is one
//                                           number or a vector)
//   y_k  = h_k + sum_j w_k[j] * h_k[t - taps + 1 + j]     (per channel; zeros before the sequence's start)
//
// The last taps - 1 rows u of a sequence are its state ("tail", 32-bit, one slot per sequence, shared by both
// sublayers because h_k differs from u by a gain only).
//
// A workgroup takes R consecutive new tokens of one sequence: its waves first reduce the rows (and the taps - 1 rows
// before them, so no workgroup waits for another), then every thread walks its columns down the rows with the last
// taps - 1 values in registers. Only the workgroup of a sequence's first new token touches the tail: it reads it
// before it writes it, and R >= taps - 1 keeps every other workgroup's history inside the step's own rows.
#include "hds_common.h"

namespace {
using namespace hds;

constexpr int kU = 4;         // loads in flight per lane and operand
constexpr int kMaxRows = 64;  // rows a workgroup holds statistics of: R + 2 (taps - 1) at most

template <typename T>
struct InputNormParams {
  const float* x;         // [T, W] 32-bit residual, or null: rows of `embed` picked by `ids`
  const T* embed;         // [vocab, W]
  const int64_t* ids;     // [T]
  const T* delta;         // [T, W] or null
  float* x_out;           // [T, W] (another buffer than x)
  const float* g[2];      // gains: one number (gs = 0) or [W] (gs = 1)
  int gs[2];
  const float* w[2];      // [taps, W] or null (no convolution)
  T* y[2];                // [T, W]; y[1] null: one output
  float* tail;            // [slots] x slot_stride floats, [taps - 1, W] of each
  int64_t slot_stride;
  const int* slots;       // [S]
  const int* seq_meta;    // [S][3] = {q_start, n_new, seen}
  int W, taps, R;
  float eps;
};

template <typename T, int V>
__device__ __forceinline__ void load_sum(const InputNormParams<T>& p, int row, int c, float (&v)[V]) {
  if (p.x != nullptr)
    VecN<float, V>::load(p.x + (int64_t)row * p.W + c, v);
  else
    VecN<T, V>::load(p.embed + p.ids[row] * (int64_t)p.W + c, v);
  if (p.delta != nullptr) {
    float d[V];
    VecN<T, V>::load(p.delta + (int64_t)row * p.W + c, d);
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] += d[i];
  }
}

// M: registers of history, >= taps - 1 (missing taps have no weight)
template <typename T, int V, int M, int NT>
__global__ __launch_bounds__(NT) void input_norm_kernel(InputNormParams<T> p) {
  __shared__ float s_rstd[kMaxRows];
  __shared__ float s_part[NT / 64];
  const int seq = blockIdx.y;
  const int q0 = p.seq_meta[3 * seq], n = p.seq_meta[3 * seq + 1], seen = p.seq_meta[3 * seq + 2];
  const int start = blockIdx.x * p.R;
  if (start >= n) return;
  const int rows = min(p.R, n - start);
  const int m = p.taps - 1;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const bool first = blockIdx.x == 0;
  const int halo = min(m, start);                 // rows before `start` that belong to this step
  // rows of the new tail that are not among this workgroup's own (statistics only)
  const int t_lo = first ? max(max(n - m, 0), rows) : n;
  const int extra = n - t_lo;
  const int total = halo + rows + extra;
  if (total == 1 && NT > 64) {  // one row: the whole workgroup reduces it
    const int row = q0 + start;
    float ss = 0.f;
    for (int c = threadIdx.x * V; c < p.W; c += NT * V) {
      float v[V];
      load_sum<T, V>(p, row, c, v);
#pragma unroll
      for (int i = 0; i < V; ++i) ss += v[i] * v[i];
      VecN<float, V>::store(p.x_out + (int64_t)row * p.W + c, v);
    }
    ss = wave_sum(ss);
    if (lane == 0) s_part[wid] = ss;
    __syncthreads();
    if (threadIdx.x == 0) {
      float a = 0.f;
      for (int i = 0; i < NT / 64; ++i) a += s_part[i];
      s_rstd[0] = 1.f / sqrtf(a / (float)p.W + p.eps);
    }
  } else {
    for (int r = wid; r < total; r += NT / 64) {
      const int i = r < halo + rows ? start - halo + r : t_lo + (r - halo - rows);  // index among the new tokens
      const bool own = r >= halo && r < halo + rows;
      const int row = q0 + i;
      float ss = 0.f;
      for (int c0 = lane * V; c0 < p.W; c0 += 64 * V * kU) {
        float v[kU][V];
#pragma unroll
        for (int k = 0; k < kU; ++k)
          if (c0 + 64 * V * k < p.W) load_sum<T, V>(p, row, c0 + 64 * V * k, v[k]);
#pragma unroll
        for (int k = 0; k < kU; ++k) {
          const int c = c0 + 64 * V * k;
          if (c >= p.W) continue;
#pragma unroll
          for (int i2 = 0; i2 < V; ++i2) ss += v[k][i2] * v[k][i2];
          if (own) VecN<float, V>::store(p.x_out + (int64_t)row * p.W + c, v[k]);
        }
      }
      ss = wave_sum(ss);
      if (lane == 0) s_rstd[r] = 1.f / sqrtf(ss / (float)p.W + p.eps);
    }
  }
  __syncthreads();
  float* tail = m > 0 ? p.tail + (int64_t)p.slots[seq] * p.slot_stride : nullptr;
  const int nout = p.y[1] != nullptr ? 2 : 1;
  for (int c = threadIdx.x * V; c < p.W; c += NT * V) {
    float hist[M > 0 ? M : 1][V];  // hist[k]: u of the row k + 1 before the current one
#pragma unroll
    for (int k = 0; k < M; ++k) {
#pragma unroll
      for (int i = 0; i < V; ++i) hist[k][i] = 0.f;
      if (k >= m) continue;
      const int i0 = start - 1 - k;
      if (i0 >= 0) {
        load_sum<T, V>(p, q0 + i0, c, hist[k]);
        const float rs = s_rstd[halo - 1 - k];
#pragma unroll
        for (int i = 0; i < V; ++i) hist[k][i] *= rs;
      } else if (seen + i0 >= 0) {  // tail entry e holds position seen - m + e
        VecN<float, V>::load(tail + (int64_t)(m + i0) * p.W + c, hist[k]);
      }
    }
    float g[2][V], w[2][M + 1][V];  // w[.][k]: the tap of the row k back
#pragma unroll
    for (int o = 0; o < 2; ++o) {
      if (o >= nout) break;
      if (p.gs[o])
        VecN<float, V>::load(p.g[o] + c, g[o]);
      else {
#pragma unroll
        for (int i = 0; i < V; ++i) g[o][i] = p.g[o][0];
      }
#pragma unroll
      for (int k = 0; k <= M; ++k) {
#pragma unroll
        for (int i = 0; i < V; ++i) w[o][k][i] = 0.f;
        if (k <= m && p.w[o] != nullptr) VecN<float, V>::load(p.w[o] + (int64_t)(m - k) * p.W + c, w[o][k]);
      }
    }
    for (int r0 = 0; r0 < rows; r0 += kU) {
      float us[kU][V];
#pragma unroll
      for (int b = 0; b < kU; ++b)
        if (r0 + b < rows) load_sum<T, V>(p, q0 + start + r0 + b, c, us[b]);
#pragma unroll
      for (int b = 0; b < kU; ++b) {
        const int r = r0 + b;
        if (r >= rows) break;
        const int row = q0 + start + r;
        float (&u)[V] = us[b];
        const float rs = s_rstd[halo + r];
#pragma unroll
        for (int i = 0; i < V; ++i) u[i] *= rs;
#pragma unroll
        for (int o = 0; o < 2; ++o) {
          if (o >= nout) break;
          float y[V];
#pragma unroll
          for (int i = 0; i < V; ++i) {
            float a = u[i] + w[o][0][i] * u[i];
#pragma unroll
            for (int k = 0; k < M; ++k) a += w[o][k + 1][i] * hist[k][i];
            y[i] = a * g[o][i];
          }
          VecN<T, V>::store(p.y[o] + (int64_t)row * p.W + c, y);
        }
#pragma unroll
        for (int k = M - 1; k > 0; --k)
#pragma unroll
          for (int i = 0; i < V; ++i) hist[k][i] = hist[k - 1][i];
        if (M > 0) {
#pragma unroll
          for (int i = 0; i < V; ++i) hist[0][i] = u[i];
        }
      }
    }
    if (first && m > 0) {
      for (int e = 0; e < m; ++e) {
        const int i0 = n - m + e;  // index among the new tokens
        float u[V];
        if (i0 >= 0) {
          load_sum<T, V>(p, q0 + i0, c, u);
          const float rs = s_rstd[i0 < rows ? i0 : rows + (i0 - t_lo)];
#pragma unroll
          for (int i = 0; i < V; ++i) u[i] *= rs;
        } else if (seen + i0 >= 0) {
          VecN<float, V>::load(tail + (int64_t)(e + n) * p.W + c, u);
        } else {
#pragma unroll
          for (int i = 0; i < V; ++i) u[i] = 0.f;
        }
        VecN<float, V>::store(tail + (int64_t)e * p.W + c, u);
      }
    }
  }
}

// One new token per sequence: a workgroup of 1024 threads a row, P * 4 columns a thread. Everything the row needs is
// requested before the reduction, so the step is one memory round trip and one barrier long.
template <typename T, int M, int P>
__global__ __launch_bounds__(1024) void input_norm_step_kernel(InputNormParams<T> p) {
  __shared__ float s_part[16];
  const int seq = blockIdx.x;
  if (p.seq_meta[3 * seq + 1] <= 0) return;
  const int row = p.seq_meta[3 * seq], seen = p.seq_meta[3 * seq + 2];
  const int m = p.taps - 1;
  float* tail = M > 0 ? p.tail + (int64_t)p.slots[seq] * p.slot_stride : nullptr;
  const int nout = p.y[1] != nullptr ? 2 : 1;
  float u[P][4], hist[P][M > 0 ? M : 1][4], w[P][2][M + 1][4], g[P][2][4];
  float ss = 0.f;
#pragma unroll
  for (int q = 0; q < P; ++q) {
    const int c = (q * 1024 + threadIdx.x) * 4;
    if (c >= p.W) continue;
    load_sum<T, 4>(p, row, c, u[q]);
#pragma unroll
    for (int k = 0; k < M; ++k) {  // hist[k]: k + 1 back; entries before the sequence's start are zero
#pragma unroll
      for (int i = 0; i < 4; ++i) hist[q][k][i] = 0.f;
      if (k < m && seen - 1 - k >= 0) VecN<float, 4>::load(tail + (int64_t)(m - 1 - k) * p.W + c, hist[q][k]);
    }
#pragma unroll
    for (int o = 0; o < 2; ++o) {
      if (o >= nout) break;
#pragma unroll
      for (int k = 0; k <= M; ++k) {
#pragma unroll
        for (int i = 0; i < 4; ++i) w[q][o][k][i] = 0.f;
        if (k <= m && p.w[o] != nullptr) VecN<float, 4>::load(p.w[o] + (int64_t)(m - k) * p.W + c, w[q][o][k]);
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) g[q][o][i] = p.g[o][p.gs[o] ? c + i : 0];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) ss += u[q][i] * u[q][i];
  }
  ss = wave_sum(ss);
  if ((threadIdx.x & 63) == 0) s_part[threadIdx.x >> 6] = ss;
  __syncthreads();
  ss = 0.f;
#pragma unroll
  for (int i = 0; i < 16; ++i) ss += s_part[i];
  const float rs = 1.f / sqrtf(ss / (float)p.W + p.eps);
#pragma unroll
  for (int q = 0; q < P; ++q) {
    const int c = (q * 1024 + threadIdx.x) * 4;
    if (c >= p.W) continue;
    VecN<float, 4>::store(p.x_out + (int64_t)row * p.W + c, u[q]);
#pragma unroll
    for (int i = 0; i < 4; ++i) u[q][i] *= rs;
#pragma unroll
    for (int o = 0; o < 2; ++o) {
      if (o >= nout) break;
      float y[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        float a = u[q][i] + w[q][o][0][i] * u[q][i];
#pragma unroll
        for (int k = 0; k < M; ++k) a += w[q][o][k + 1][i] * hist[q][k][i];
        y[i] = a * g[q][o][i];
      }
      VecN<T, 4>::store(p.y[o] + (int64_t)row * p.W + c, y);
    }
#pragma unroll
    for (int k = 0; k < M; ++k)
      if (k < m) VecN<float, 4>::store(tail + (int64_t)(m - 1 - k) * p.W + c, k == 0 ? u[q] : hist[q][k > 0 ? k - 1 : 0]);
  }
}

template <typename T, int V, int NT>
int launch_input_norm(const InputNormParams<T>& p, int n_seqs, int max_new, hipStream_t st) {
  const dim3 grid((max_new + p.R - 1) / p.R, n_seqs);
  const int m = p.taps - 1;
  if constexpr (V == 1) {
    if (m > 3) {
      if (m <= 7) hipLaunchKernelGGL((input_norm_kernel<T, 1, 7, NT>), grid, dim3(NT), 0, st, p);
      else hipLaunchKernelGGL((input_norm_kernel<T, 1, 15, NT>), grid, dim3(NT), 0, st, p);
      return hipGetLastError();
    }
  }
#define HDS_IN(MM) hipLaunchKernelGGL((input_norm_kernel<T, V, MM, NT>), grid, dim3(NT), 0, st, p)
  if (m == 0) HDS_IN(0);
  else if (m == 1) HDS_IN(1);
  else if (m == 2) HDS_IN(2);
  else HDS_IN(3);
#undef HDS_IN
  return hipGetLastError();
}

template <typename T>
int input_norm(const InputNormParams<T>& p, int n_seqs, int max_new, hipStream_t st) {
  const bool v4 = p.W % 4 == 0 && p.slot_stride % 4 == 0;
  if (max_new == 1 && v4 && p.taps <= 4 && p.W <= 8192) {
#define HDS_IS(MM)                                                                                              \
  if (p.W <= 4096) hipLaunchKernelGGL((input_norm_step_kernel<T, MM, 1>), dim3(n_seqs), dim3(1024), 0, st, p); \
  else hipLaunchKernelGGL((input_norm_step_kernel<T, MM, 2>), dim3(n_seqs), dim3(1024), 0, st, p)
    if (p.taps == 1) { HDS_IS(0); } else if (p.taps == 2) { HDS_IS(1); } else if (p.taps == 3) { HDS_IS(2); } else { HDS_IS(3); }
#undef HDS_IS
    return hipGetLastError();
  }
  if (v4 && p.taps <= 4) return launch_input_norm<T, 4, 512>(p, n_seqs, max_new, st);
  return launch_input_norm<T, 1, 256>(p, n_seqs, max_new, st);
}

}  // namespace

// taps: 1 .. 16; R: new tokens per workgroup, >= taps - 1 unless max_new == 1, and R + 2 (taps - 1) <= 64. seq_meta /
// slots describe the step's sequences; every sequence has at most max_new new tokens. Vectors must be 16-B aligned when
// W % 4 == 0.
HDS_EXPORT int hds_input_norm(int dtype, const float* x, const void* embed, const int64_t* ids, const void* delta,
                              float* x_out, const float* g0, int gs0, const float* w0, void* y0, const float* g1,
                              int gs1, const float* w1, void* y1, float* tail, int64_t slot_stride, const int* slots,
                              const int* seq_meta, int n_seqs, int max_new, int W, int taps, int R, float eps,
                              hipStream_t st) {
  if (n_seqs <= 0 || max_new <= 0) return 0;
  if (W < 1 || taps < 1 || taps > 16 || R < 1 || (max_new > 1 && R < taps - 1) || R + 2 * (taps - 1) > kMaxRows ||
      (x == nullptr && (embed == nullptr || ids == nullptr)) || x == x_out || n_seqs > 65535 ||
      (taps > 1 && (tail == nullptr || slots == nullptr)) || y0 == nullptr || g0 == nullptr ||
      (y1 != nullptr && g1 == nullptr))
    return hipErrorInvalidValue;
  if (dtype == kBF16) {
    InputNormParams<bf16> p{x, (const bf16*)embed, ids, (const bf16*)delta, x_out, {g0, g1}, {gs0, gs1}, {w0, w1},
                            {(bf16*)y0, (bf16*)y1}, tail, slot_stride, slots, seq_meta, W, taps, R, eps};
    return input_norm(p, n_seqs, max_new, st);
  }
  if (dtype == kF32) {
    InputNormParams<float> p{x, (const float*)embed, ids, (const float*)delta, x_out, {g0, g1}, {gs0, gs1}, {w0, w1},
                             {(float*)y0, (float*)y1}, tail, slot_stride, slots, seq_meta, W, taps, R, eps};
    return input_norm(p, n_seqs, max_new, st);
  }
  return hipErrorInvalidValue;
}
