// Gated linear recurrence of a recurrent mixer (minGRU): element by element over time, in 32-bit,
//
//   z = sigmoid(a + ba),  u = b + bb,  v = u + 1/2 (u >= 0) or sigmoid(u) (u < 0)
//   S_t = (1 - z) S_(t-1) + z v,       out_t = S_t * silu(c)
//
// with a | b | c the three column blocks of one projection row. The state of a sequence is one 32-bit row in its slot;
// a sequence whose `seen` is 0 starts from zero whatever the slot holds.
//
// Short steps (decode, small portions) run one thread per V channels over the new tokens. Longer portions run a
// workgroup per 16 channels: 64 thread groups take G consecutive tokens each, keep their gates in registers, compose
// them to one map S -> A S + B, find the state they start from over the wave (shuffles) and the workgroup (LDS), and
// write their outputs. Every value is read and every gate evaluated once; the next 64 G tokens are requested before
// this step's are worked on.
#include "hds_common.h"

namespace {
using namespace hds;

template <typename T, int V>
__device__ __forceinline__ void ldv(const T* p, float (&v)[V]) {
  if constexpr (V == 1) {
    v[0] = to_f(*p);
  } else if constexpr (sizeof(T) == 2) {
    const bf16x4 r = *reinterpret_cast<const bf16x4*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = (float)r[i];
  } else {
    const f32x4 r = *reinterpret_cast<const f32x4*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = r[i];
  }
}
template <typename T, int V>
__device__ __forceinline__ void stv(T* p, const float (&v)[V]) {
  if constexpr (V == 1) {
    *p = from_f<T>(v[0]);
  } else if constexpr (sizeof(T) == 2) {
    bf16x4 r;
#pragma unroll
    for (int i = 0; i < 4; ++i) r[i] = (bf16)v[i];
    *reinterpret_cast<bf16x4*>(p) = r;
  } else {
    *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
  }
}

__device__ __forceinline__ float exp_neg_abs(float x) { return __builtin_amdgcn_exp2f(-1.4426950408889634f * fabsf(x)); }

// 1 - z, z * v and g * sigmoid(g). Every sigmoid is 1 / (1 + e) or e / (1 + e) with e = exp(-|x|) <= 1 (no
// cancellation, no overflow); one reciprocal of the product of the 1 + e serves all three.
__device__ __forceinline__ void gates(float a, float b, float g, float& keep, float& add, float& og) {
  const float ea = exp_neg_abs(a), eb = exp_neg_abs(b), eg = exp_neg_abs(g);
  const float pa = 1.f + ea, pb = 1.f + eb, pg = 1.f + eg;
  const float r = __builtin_amdgcn_rcpf(pa * pb * pg);
  const float ra = r * (pb * pg), rb = r * (pa * pg), rg = g * (r * (pa * pb));
  keep = a >= 0.f ? ea * ra : ra;
  add = (a >= 0.f ? ra : ea * ra) * (b >= 0.f ? b + 0.5f : eb * rb);
  og = g >= 0.f ? rg : eg * rg;
}

template <typename T>
struct ScanParams {
  const T* in;       // [tokens, ld]: a at column 0, b at W, c at 2 W
  int64_t ld;
  const float* ba;   // [W]
  const float* bb;
  T* out;            // [tokens, ldo]
  int64_t ldo;
  float* state;      // [slots] x slot_stride
  int64_t slot_stride;
  const int* slots;
  const int* seq_meta;
  int W;
};

template <typename T, int V>
__global__ __launch_bounds__(64) void scan_serial_kernel(ScanParams<T> p) {
  const int c = (blockIdx.x * 64 + threadIdx.x) * V;
  if (c >= p.W) return;
  const int seq = blockIdx.y;
  const int q0 = p.seq_meta[3 * seq], n = p.seq_meta[3 * seq + 1], seen = p.seq_meta[3 * seq + 2];
  float ba[V], bb[V], s[V];
  ldv<float, V>(p.ba + c, ba);
  ldv<float, V>(p.bb + c, bb);
  float* st = p.state + (int64_t)p.slots[seq] * p.slot_stride + c;
#pragma unroll
  for (int i = 0; i < V; ++i) s[i] = 0.f;
  if (seen > 0) ldv<float, V>(st, s);
  constexpr int U = 4;
  for (int t = 0; t < n; t += U) {
    float a[U][V], b[U][V], g[U][V];
#pragma unroll
    for (int k = 0; k < U; ++k)
      if (t + k < n) {
        const T* in = p.in + (int64_t)(q0 + t + k) * p.ld + c;
        ldv<T, V>(in, a[k]);
        ldv<T, V>(in + p.W, b[k]);
        ldv<T, V>(in + 2 * p.W, g[k]);
      }
#pragma unroll
    for (int k = 0; k < U; ++k) {
      if (t + k >= n) break;
      float y[V];
#pragma unroll
      for (int i = 0; i < V; ++i) {
        float keep, add, og;
        gates(a[k][i] + ba[i], b[k][i] + bb[i], g[k][i], keep, add, og);
        s[i] = keep * s[i] + add;
        y[i] = s[i] * og;
      }
      stv<T, V>(p.out + (int64_t)(q0 + t + k) * p.ldo + c, y);
    }
  }
  if (n > 0) stv<float, V>(st, s);
}

constexpr int kCols = 16, kThreads = 1024;  // channels and threads of a workgroup

// one channel and G consecutive tokens a thread; row offsets of a sequence fit 32 bits
template <typename T, int G>
__global__ __launch_bounds__(kThreads) void scan_block_kernel(ScanParams<T> p) {
  constexpr int NW = kThreads / 64, STEP = kThreads / kCols * G;
  __shared__ float sA[2][NW][kCols], sB[2][NW][kCols];
  // neighbouring channel blocks share cache lines: keep them on one XCD (workgroups go round-robin over the 8)
  const int nb = gridDim.x, bx = nb % 8 == 0 ? (blockIdx.x & 7) * (nb / 8) + (blockIdx.x >> 3) : blockIdx.x;
  const int cl = threadIdx.x & (kCols - 1), grp = threadIdx.x / kCols;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const bool ok = bx * kCols + cl < p.W;
  const int c = ok ? bx * kCols + cl : p.W - 1;
  const int seq = blockIdx.y;
  const int q0 = p.seq_meta[3 * seq], n = p.seq_meta[3 * seq + 1], seen = p.seq_meta[3 * seq + 2];
  if (n <= 0) return;
  float* st = p.state + (int64_t)p.slots[seq] * p.slot_stride + c;
  const float ba = p.ba[c], bb = p.bb[c];
  float s = seen > 0 ? *st : 0.f;  // the state before this step, the same in every thread of a channel
  const T* in_a = p.in + (int64_t)q0 * p.ld;
  const T* in_b = in_a + p.W;
  const T* in_g = in_b + p.W;
  T* out = p.out + (int64_t)q0 * p.ldo;
  const uint32_t ld = (uint32_t)p.ld, ldo = (uint32_t)p.ldo;
  T ra[G], rb[G], rg[G];
  auto fetch = [&](int t0) {
    const int t = t0 + grp * G;
    const bool full = t0 + STEP <= n;
    uint32_t o = (uint32_t)t * ld + c;
#pragma unroll
    for (int k = 0; k < G; ++k) {
      if (!full) o = (uint32_t)min(t + k, n - 1) * ld + c;
      ra[k] = in_a[o];
      rb[k] = in_b[o];
      rg[k] = in_g[o];
      o += ld;
    }
  };
  fetch(0);
  for (int t0 = 0, it = 0; t0 < n; t0 += STEP, ++it) {
    const int left = n - (t0 + grp * G);  // tokens this thread has
    float keep[G], add[G], og[G];
    float A = 1.f, B = 0.f;
#pragma unroll
    for (int k = 0; k < G; ++k) {
      gates(to_f(ra[k]) + ba, to_f(rb[k]) + bb, to_f(rg[k]), keep[k], add[k], og[k]);
      if (k >= left) {
        keep[k] = 1.f;
        add[k] = 0.f;
      }
      B = keep[k] * B + add[k];
      A *= keep[k];
    }
    if (t0 + STEP < n) fetch(t0 + STEP);
    // inclusive composition over the wave's four groups
#pragma unroll
    for (int d = kCols; d < 64; d <<= 1) {
      const float pa = __shfl_up(A, d, 64), pb = __shfl_up(B, d, 64);
      if (lane >= d) {
        B = A * pb + B;
        A *= pa;
      }
    }
    const int buf = it & 1;
    if (lane >= 64 - kCols) {
      sA[buf][w][cl] = A;
      sB[buf][w][cl] = B;
    }
    float ea = __shfl_up(A, kCols, 64), eb = __shfl_up(B, kCols, 64);
    if (lane < kCols) {
      ea = 1.f;
      eb = 0.f;
    }
    __syncthreads();  // one barrier a step: the other buffer is written next
    float sw = s;
#pragma unroll 4
    for (int i = 0; i < NW; ++i) {
      if (i == w) sw = s;
      s = sA[buf][i][cl] * s + sB[buf][i][cl];
    }
    float cur = ea * sw + eb;
    uint32_t o = (uint32_t)(t0 + grp * G) * ldo + c;
#pragma unroll
    for (int k = 0; k < G; ++k) {
      cur = keep[k] * cur + add[k];
      if (ok && k < left) out[o] = from_f<T>(cur * og[k]);
      o += ldo;
    }
  }
  if (ok && grp == 0) *st = s;
}

template <typename T>
int scan(const ScanParams<T>& p, int n_seqs, int max_new, hipStream_t st) {
  // (steps whose rows span 2^31 bytes and more: one thread per channel, 64-bit offsets)
  const int64_t span = (int64_t)max_new * (p.ld > p.ldo ? p.ld : p.ldo) * (int64_t)sizeof(T);
  if (max_new > 32 && span < (int64_t)0x7fffffff) {
    const dim3 grid((p.W + kCols - 1) / kCols, n_seqs);
    if (max_new <= 1024)
      hipLaunchKernelGGL((scan_block_kernel<T, 4>), grid, dim3(kThreads), 0, st, p);
    else
      hipLaunchKernelGGL((scan_block_kernel<T, 8>), grid, dim3(kThreads), 0, st, p);
    return hipGetLastError();
  }
  if (p.W % 4 == 0 && p.ld % 4 == 0 && p.ldo % 4 == 0 && p.slot_stride % 4 == 0 && (uintptr_t)p.in % 16 == 0 &&
      (uintptr_t)p.out % 16 == 0 && (uintptr_t)p.state % 16 == 0)
    hipLaunchKernelGGL((scan_serial_kernel<T, 4>), dim3((p.W + 255) / 256, n_seqs), dim3(64), 0, st, p);
  else
    hipLaunchKernelGGL((scan_serial_kernel<T, 1>), dim3((p.W + 63) / 64, n_seqs), dim3(64), 0, st, p);
  return hipGetLastError();
}

}  // namespace

HDS_EXPORT int hds_gated_scan(int dtype, const void* in, int64_t ld, const float* ba, const float* bb, void* out,
                              int64_t ldo, float* state, int64_t slot_stride, const int* slots, const int* seq_meta,
                              int n_seqs, int max_new, int W, hipStream_t st) {
  if (n_seqs <= 0 || max_new <= 0) return 0;
  if (W < 1 || ld < 3 * (int64_t)W || ldo < W || !state || !slots || n_seqs > 65535) return hipErrorInvalidValue;
  if (dtype == kBF16) {
    ScanParams<bf16> p{(const bf16*)in, ld, ba, bb, (bf16*)out, ldo, state, slot_stride, slots, seq_meta, W};
    return scan(p, n_seqs, max_new, st);
  }
  if (dtype == kF32) {
    ScanParams<float> p{(const float*)in, ld, ba, bb, (float*)out, ldo, state, slot_stride, slots, seq_meta, W};
    return scan(p, n_seqs, max_new, st);
  }
  return hipErrorInvalidValue;
}
