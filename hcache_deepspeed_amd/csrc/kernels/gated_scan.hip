// Gated linear recurrence of a recurrent mixer (minGRU): element by element over time, in 32-bit,
//
//   z = sigmoid(a + ba),  u = b + bb,  v = u + 1/2 (u >= 0) or sigmoid(u) (u < 0)
//   S_t = (1 - z) S_(t-1) + z v,       out_t = S_t * silu(c)
//
// with a | b | c the three column blocks of one projection row. The state of a sequence is one 32-bit row in its slot;
// a sequence whose `seen` is 0 starts from zero whatever the slot holds.
//
// Short steps (decode, small portions) run one thread per channel over the new tokens. Prompts are cut into chunks of
// kChunk tokens: pass 1 reduces every chunk to S_out = A S_in + B, pass 2 composes the chunks of a sequence and leaves
// each chunk's S_in (and the sequence's new state), pass 3 replays the chunks from it. No workgroup waits for another.
#include "hds_common.h"

namespace {
using namespace hds;

constexpr int kChunk = 32;
typedef __bf16 bf16x2 __attribute__((ext_vector_type(2)));

template <typename T, int V>
__device__ __forceinline__ void ldv(const T* p, float (&v)[V]) {
  if constexpr (V == 1) {
    v[0] = to_f(*p);
  } else if constexpr (V == 2 && sizeof(T) == 2) {
    const bf16x2 r = *reinterpret_cast<const bf16x2*>(p);
    v[0] = (float)r[0];
    v[1] = (float)r[1];
  } else if constexpr (V == 2) {
    const float2 r = *reinterpret_cast<const float2*>(p);
    v[0] = r.x;
    v[1] = r.y;
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
  } else if constexpr (V == 2 && sizeof(T) == 2) {
    *reinterpret_cast<bf16x2*>(p) = bf16x2{(bf16)v[0], (bf16)v[1]};
  } else if constexpr (V == 2) {
    *reinterpret_cast<float2*>(p) = make_float2(v[0], v[1]);
  } else if constexpr (sizeof(T) == 2) {
    bf16x4 r;
#pragma unroll
    for (int i = 0; i < 4; ++i) r[i] = (bf16)v[i];
    *reinterpret_cast<bf16x4*>(p) = r;
  } else {
    *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
  }
}

// 1 - z, z * v and (with OUT) g * sigmoid(g). Every sigmoid is 1 / (1 + e) or e / (1 + e) with e = exp(-|x|) <= 1 (no
// cancellation, no overflow); one reciprocal of the product of the 1 + e serves all of them.
template <bool OUT>
__device__ __forceinline__ void gates(float a, float b, float g, float& keep, float& add, float& og) {
  const float ea = __expf(-fabsf(a)), eb = __expf(-fabsf(b)), eg = OUT ? __expf(-fabsf(g)) : 0.f;
  const float pa = 1.f + ea, pb = 1.f + eb, pg = 1.f + eg;
  const float r = __builtin_amdgcn_rcpf(OUT ? pa * pb * pg : pa * pb);
  const float ra = OUT ? r * (pb * pg) : r * pb;
  const float rb = OUT ? r * (pa * pg) : r * pa;
  keep = a >= 0.f ? ea * ra : ra;
  const float z = a >= 0.f ? ra : ea * ra;
  add = z * (b >= 0.f ? b + 0.5f : eb * rb);
  if (OUT) {
    const float rg = g * (r * (pa * pb));
    og = g >= 0.f ? rg : eg * rg;
  }
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
  float* ws;         // [S, W / V, chunks, 2 V]: A then B (after pass 2: the chunk's S_in) of V channels
  int W, chunks;
};

// pass 0: whole sequences serially; pass 1: chunk reductions; pass 3: chunk replays
template <typename T, int V, int PASS>
__global__ __launch_bounds__(64) void scan_kernel(ScanParams<T> p) {
  const int c = (blockIdx.x * 64 + threadIdx.x) * V;
  if (c >= p.W) return;
  const int seq = blockIdx.z, ch = blockIdx.y;
  const int q0 = p.seq_meta[3 * seq], n = p.seq_meta[3 * seq + 1], seen = p.seq_meta[3 * seq + 2];
  const int t0 = PASS == 0 ? 0 : ch * kChunk;
  if (t0 >= n) return;
  const int t1 = PASS == 0 ? n : min(n, t0 + kChunk);
  float ba[V], bb[V], s[V], A[V];
  ldv<float, V>(p.ba + c, ba);
  ldv<float, V>(p.bb + c, bb);
  float* st = p.state + (PASS == 0 ? (int64_t)p.slots[seq] * p.slot_stride + c : 0);
  float* ws = PASS == 0 ? nullptr : p.ws + (((int64_t)seq * (p.W / V) + c / V) * p.chunks + ch) * (2 * V);
#pragma unroll
  for (int i = 0; i < V; ++i) {
    s[i] = 0.f;
    A[i] = 1.f;
  }
  if (PASS == 0 && seen > 0) ldv<float, V>(st, s);
  if (PASS == 3) ldv<float, V>(ws + V, s);
  const T* in = p.in + (int64_t)(q0 + t0) * p.ld + c;
  T* out = p.out + (int64_t)(q0 + t0) * p.ldo + c;
  auto step = [&](const float (&a)[V], const float (&b)[V], const float (&g)[V], T* o) {
    float y[V];
#pragma unroll
    for (int i = 0; i < V; ++i) {
      float keep, add, og;
      gates<PASS != 1>(a[i] + ba[i], b[i] + bb[i], g[i], keep, add, og);
      s[i] = keep * s[i] + add;
      if (PASS == 1) A[i] *= keep;
      if (PASS != 1) y[i] = s[i] * og;
    }
    if (PASS != 1) stv<T, V>(o, y);
  };
  constexpr int U = 8;
  int t = t0;
  for (; t + U <= t1; t += U) {
    float a[U][V], b[U][V], g[U][V];
#pragma unroll
    for (int k = 0; k < U; ++k) {
      ldv<T, V>(in + k * p.ld, a[k]);
      ldv<T, V>(in + k * p.ld + p.W, b[k]);
      if (PASS != 1) ldv<T, V>(in + k * p.ld + 2 * p.W, g[k]);
    }
#pragma unroll
    for (int k = 0; k < U; ++k) step(a[k], b[k], g[k], out + k * p.ldo);
    in += U * p.ld;
    out += U * p.ldo;
  }
  for (; t < t1; ++t) {
    float a[V], b[V], g[V];
    ldv<T, V>(in, a);
    ldv<T, V>(in + p.W, b);
    if (PASS != 1) ldv<T, V>(in + 2 * p.W, g);
    step(a, b, g, out);
    in += p.ld;
    out += p.ldo;
  }
  if (PASS == 0) stv<float, V>(st, s);
  if (PASS == 1) {
    stv<float, V>(ws, A);
    stv<float, V>(ws + V, s);
  }
}

// pass 2: a wave per V channels of a sequence, a chunk per lane: prefix composition of the chunks' maps S -> A S + B by
// shuffles, 64 chunks at a time; every chunk's S_in goes back to ws, the last state to the sequence's slot
template <typename T, int V>
__global__ __launch_bounds__(64) void scan_carry_kernel(ScanParams<T> p) {
  const int c = blockIdx.x * V, lane = threadIdx.x;
  const int seq = blockIdx.y;
  const int n = p.seq_meta[3 * seq + 1], seen = p.seq_meta[3 * seq + 2];
  if (n <= 0) return;
  const int nc = (n + kChunk - 1) / kChunk;
  float* st = p.state + (int64_t)p.slots[seq] * p.slot_stride + c;
  float s[V];
#pragma unroll
  for (int i = 0; i < V; ++i) s[i] = 0.f;
  if (seen > 0) ldv<float, V>(st, s);
  float* ws = p.ws + ((int64_t)seq * (p.W / V) + blockIdx.x) * p.chunks * (2 * V);
  for (int k0 = 0; k0 < nc; k0 += 64) {
    const int k = k0 + lane;
    float A[V], B[V], in[V];
#pragma unroll
    for (int i = 0; i < V; ++i) {
      A[i] = 1.f;
      B[i] = 0.f;
    }
    if (k < nc) {
      ldv<float, V>(ws + (int64_t)k * 2 * V, A);
      ldv<float, V>(ws + (int64_t)k * 2 * V + V, B);
    }
#pragma unroll
    for (int i = 0; i < V; ++i) {
#pragma unroll
      for (int d = 1; d < 64; d <<= 1) {
        const float pa = __shfl_up(A[i], d, 64), pb = __shfl_up(B[i], d, 64);
        if (lane >= d) {
          B[i] = A[i] * pb + B[i];
          A[i] *= pa;
        }
      }
      const float ea = __shfl_up(A[i], 1, 64), eb = __shfl_up(B[i], 1, 64);
      in[i] = lane == 0 ? s[i] : ea * s[i] + eb;
      s[i] = __shfl(A[i], 63, 64) * s[i] + __shfl(B[i], 63, 64);
    }
    if (k < nc) stv<float, V>(ws + (int64_t)k * 2 * V + V, in);
  }
  if (lane == 0) stv<float, V>(st, s);
}

template <typename T, int V>
int launch_scan(const ScanParams<T>& p, int n_seqs, int max_new, hipStream_t st) {
  const int cb = (p.W + 64 * V - 1) / (64 * V);
  if (p.ws == nullptr) {
    hipLaunchKernelGGL((scan_kernel<T, V, 0>), dim3(cb, 1, n_seqs), dim3(64), 0, st, p);
    return hipGetLastError();
  }
  const dim3 grid(cb, (max_new + kChunk - 1) / kChunk, n_seqs);
  hipLaunchKernelGGL((scan_kernel<T, V, 1>), grid, dim3(64), 0, st, p);
  hipLaunchKernelGGL((scan_carry_kernel<T, V>), dim3(p.W / V, n_seqs), dim3(64), 0, st, p);
  hipLaunchKernelGGL((scan_kernel<T, V, 3>), grid, dim3(64), 0, st, p);
  return hipGetLastError();
}

template <typename T>
int scan(const ScanParams<T>& p, int n_seqs, int max_new, hipStream_t st) {
  if (p.W % 4 == 0 && p.ld % 4 == 0 && p.ldo % 4 == 0 && p.slot_stride % 4 == 0 && (uintptr_t)p.in % 16 == 0 &&
      (uintptr_t)p.out % 16 == 0 && (uintptr_t)p.state % 16 == 0)
    return p.ws == nullptr ? launch_scan<T, 4>(p, n_seqs, max_new, st) : launch_scan<T, 2>(p, n_seqs, max_new, st);
  return launch_scan<T, 1>(p, n_seqs, max_new, st);
}

}  // namespace

HDS_EXPORT int hds_gated_scan_chunk() { return kChunk; }

// ws: null -> every sequence serially; else n_seqs * chunks * 2 * W floats with chunks = ceil(max_new / kChunk)
HDS_EXPORT int hds_gated_scan(int dtype, const void* in, int64_t ld, const float* ba, const float* bb, void* out,
                              int64_t ldo, float* state, int64_t slot_stride, const int* slots, const int* seq_meta,
                              float* ws, int n_seqs, int max_new, int W, hipStream_t st) {
  if (n_seqs <= 0 || max_new <= 0) return 0;
  if (W < 1 || ld < 3 * (int64_t)W || ldo < W || !state || !slots || n_seqs > 65535) return hipErrorInvalidValue;
  const int chunks = (max_new + kChunk - 1) / kChunk;
  if (chunks > 65535) return hipErrorInvalidValue;
  if (dtype == kBF16) {
    ScanParams<bf16> p{(const bf16*)in, ld, ba, bb, (bf16*)out, ldo, state, slot_stride, slots, seq_meta, ws, W, chunks};
    return scan(p, n_seqs, max_new, st);
  }
  if (dtype == kF32) {
    ScanParams<float> p{(const float*)in, ld, ba, bb, (float*)out, ldo, state, slot_stride, slots, seq_meta, ws, W,
                        chunks};
    return scan(p, n_seqs, max_new, st);
  }
  return hipErrorInvalidValue;
}
