// What lies between the q / k / v projection and paged attention for heads with short convolutions, norms over whole
// projections and rotation:
//
//   u = conv(x)                                 q and k channels: causal, depthwise, `taps` wide
//   q, k = rot(u / sqrt(mean(u^2) + eps) * w)   the mean runs over all heads of q (of k); neighbouring pairs of the first
//                                               `rot` dimensions of a head turn
//   v = u of the keys, or the projection's own value columns
//
// q goes to a matrix of its own (neighbouring rows still read the projection), k and v into the paged cache. A sequence's slot
// holds the convolution's last inputs as a ring: the input of position p is entry p % taps, [taps, C], C = (hq + hkv) dk. With
// taps - 1 of them in use, a lone token writes another entry than those it reads. A sequence whose `seen` is 0 starts from
// zero whatever the slot holds.
//
// Steps of lone tokens run a workgroup per token (head_prep8). Portions run a workgroup per run of tokens, which keeps the
// convolution's weights and its last inputs in registers (head_prep_run); sizes it does not take go token by token
// (head_prep8, head_prep) and write their ring entries in a kernel of their own (head_tail).
//
// With the heads spread over several ranks the norms need the ranks' sums: sums_out receives this rank's sums of squares
// (nothing else is written then), sums_in brings the total ones.
#include "hds_common.h"

namespace {
using namespace hds;

template <typename T>
struct PrepParams {
  const T* x;  // [tokens, ld]: q [hq dk] | k [hkv dk] | v [hkv dv] unless the keys are the values
  int64_t ld;
  int hq, hkv, dk, dv, taps, rot, shared;  // shared: the values are the keys (dv == dk)
  const float* cw;   // [taps, C], the last row is the current token's; null with taps == 1: no convolution
  const float* qn;   // [hq dk] or null: no norms
  const float* kn;   // [hkv dk]
  const float* cos_t;  // [positions, rot / 2]
  const float* sin_t;
  T* q;              // [tokens, ldq]
  int64_t ldq;
  T* cache;          // [blocks, block_size, hkv dk | hkv dv]
  const int* tables;
  int max_blocks, block_size;
  const int* tok_seq;
  const int* tok_pos;
  const int* seq_meta;  // [sequences][3] = {first row, new tokens, seen}
  float* state;
  int64_t slot_stride;
  const int* slots;
  float* sums_out;   // [tokens, 2]
  const float* sums_in;
  int width_q, width_k;  // elements the sums run over (all ranks')
  float eps;
  int n_tok;
  __device__ __host__ __forceinline__ int C() const { return (hq + hkv) * dk; }
};

template <typename T>
struct Token {
  int row, pos, q0, n;
  float* ring;
  T* slot;
};
template <typename T>
__device__ __forceinline__ Token<T> token_of(const PrepParams<T>& p, int t) {
  const int s = p.tok_seq[t], pos = p.tok_pos[t];
  const int blk = p.tables[(int64_t)s * p.max_blocks + pos / p.block_size];
  return {t, pos, p.seq_meta[3 * s], p.seq_meta[3 * s + 1],
          p.taps > 1 ? p.state + (int64_t)p.slots[s] * p.slot_stride : nullptr,
          p.cache + ((int64_t)blk * p.block_size + pos % p.block_size) * p.hkv * (p.dk + p.dv)};
}

// V convolved channels from c
template <typename T, int V>
__device__ __forceinline__ void convolve(const PrepParams<T>& p, const Token<T>& k, int c, float (&u)[V]) {
  const T* in = p.x + (int64_t)k.row * p.ld + c;
  VecN<T, V>::load(in, u);
  if (p.cw == nullptr) return;
  const int C = p.C();
  if (p.taps > 1 && k.n == 1) VecN<float, V>::store(k.ring + (int64_t)(k.pos % p.taps) * C + c, u);
  float w[V];
  VecN<float, V>::load(p.cw + (int64_t)(p.taps - 1) * C + c, w);
#pragma unroll
  for (int i = 0; i < V; ++i) u[i] *= w[i];
  const int back = min(p.taps - 1, k.pos);
#pragma unroll 3
  for (int j = 1; j <= back; ++j) {
    float h[V];
    VecN<float, V>::load(p.cw + (int64_t)(p.taps - 1 - j) * C + c, w);
    if (k.row - j >= k.q0) VecN<T, V>::load(in - (int64_t)j * p.ld, h);
    else VecN<float, V>::load(k.ring + (int64_t)((k.pos - j) % p.taps) * C + c, h);
#pragma unroll
    for (int i = 0; i < V; ++i) u[i] += w[i] * h[i];
  }
}

// sums over the q and over the k channels, in every thread; one barrier
template <int NT>
__device__ __forceinline__ void two_sums(float& a, float& b, float (*red)[NT / 64]) {
  a = wave_sum(a);
  b = wave_sum(b);
  if ((threadIdx.x & 63) == 0) {
    red[0][threadIdx.x >> 6] = a;
    red[1][threadIdx.x >> 6] = b;
  }
  __syncthreads();
  a = b = 0.f;
#pragma unroll
  for (int i = 0; i < NT / 64; ++i) {
    a += red[0][i];
    b += red[1][i];
  }
}

template <typename T>
__device__ __forceinline__ void norm_factors(const PrepParams<T>& p, const Token<T>& k, float sq, float sk, float& rq,
                                             float& rk) {
  if (p.sums_in != nullptr) {
    sq = p.sums_in[2 * (int64_t)k.row];
    sk = p.sums_in[2 * (int64_t)k.row + 1];
  }
  rq = p.qn != nullptr ? 1.f / sqrtf(sq / (float)p.width_q + p.eps) : 1.f;
  rk = p.qn != nullptr ? 1.f / sqrtf(sk / (float)p.width_k + p.eps) : 1.f;
}

// one workgroup a token, at most NC * 8 * NT channels in registers (dk, dv, ld, ldq multiples of 8)
template <typename T, int NC, int NT>
__global__ __launch_bounds__(NT) void head_prep8_kernel(PrepParams<T> p) {
  __shared__ float red[2][NT / 64];
  const Token<T> k = token_of(p, blockIdx.x);
  const int C = p.C(), cq = p.hq * p.dk;
  float u[NC][8], sq = 0.f, sk = 0.f;
#pragma unroll
  for (int x = 0; x < NC; ++x) {
    const int c = 8 * (x * NT + threadIdx.x);
    if (c >= C) continue;
    convolve<T, 8>(p, k, c, u[x]);
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) ss += u[x][i] * u[x][i];
    if (c < cq) sq += ss; else sk += ss;
  }
  if (p.qn != nullptr && p.sums_in == nullptr) two_sums<NT>(sq, sk, red);
  if (p.sums_out != nullptr) {
    if (threadIdx.x < 2) p.sums_out[2 * (int64_t)k.row + threadIdx.x] = threadIdx.x == 0 ? sq : sk;
    return;
  }
  float rq, rk;
  norm_factors(p, k, sq, sk, rq, rk);
  const int half = p.rot / 2;
#pragma unroll
  for (int x = 0; x < NC; ++x) {
    const int c = 8 * (x * NT + threadIdx.x);
    if (c >= C) continue;
    const bool is_k = c >= cq;
    if (is_k && p.shared) Vec8<T>::store(k.slot + p.hkv * p.dk + c - cq, u[x]);
    if (p.qn != nullptr) {
      float n[8];
      Vec8<float>::load(is_k ? p.kn + c - cq : p.qn + c, n);
#pragma unroll
      for (int i = 0; i < 8; ++i) u[x][i] *= (is_k ? rk : rq) * n[i];
    }
    const int e = c % p.dk / 2;  // pair
    if (e < half) {
      const float* cp = p.cos_t + (int64_t)k.pos * half + e;
      const float* sp = p.sin_t + (int64_t)k.pos * half + e;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const bool on = e + j < half;
        const float cs = on ? cp[j] : 1.f, sn = on ? sp[j] : 0.f;
        const float a = u[x][2 * j], b = u[x][2 * j + 1];
        u[x][2 * j] = a * cs - b * sn;
        u[x][2 * j + 1] = b * cs + a * sn;
      }
    }
    Vec8<T>::store(is_k ? k.slot + c - cq : p.q + (int64_t)k.row * p.ldq + c, u[x]);
  }
  if (!p.shared)
    for (int c = 8 * threadIdx.x; c < p.hkv * p.dv; c += 8 * NT) {
      float v[8];
      Vec8<T>::load(p.x + (int64_t)k.row * p.ld + C + c, v);
      Vec8<T>::store(k.slot + p.hkv * p.dk + c, v);
    }
}

// V elements as they lie in memory
template <typename T, int V>
struct Raw {
  static constexpr int N = V * sizeof(T) / 16;
  u32x4 r[N];
  __device__ __forceinline__ void load(const T* p) {
#pragma unroll
    for (int i = 0; i < N; ++i) r[i] = reinterpret_cast<const u32x4*>(p)[i];
  }
  __device__ __forceinline__ float operator[](int i) const {
    // (a copy first: a bit cast of a vector's element as such reads the vector's first)
    const uint32_t v = sizeof(T) == 4 ? r[i / 4][i % 4] : r[i / 8][i / 2 % 4];
    if constexpr (sizeof(T) == 4) return __builtin_bit_cast(float, v);
    else return __builtin_bit_cast(float, i & 1 ? v & 0xFFFF0000u : v << 16);
  }
};

// A workgroup per R >= taps - 1 tokens of a sequence, one at a time, 8 channels a thread (C <= 8 NT), M >= taps - 1. The
// workgroup of a sequence's first tokens is the only one that reads the ring, and writes it last. OCC: waves a SIMD has room for.
template <typename T, int NT, int M, int OCC>
__global__ __launch_bounds__(NT, OCC) void head_prep_run_kernel(PrepParams<T> p, int R) {
  constexpr int NW = NT / 64;
  __shared__ float red[2][2][NW];
  const int s = blockIdx.y, q0 = p.seq_meta[3 * s], n = p.seq_meta[3 * s + 1], seen = p.seq_meta[3 * s + 2];
  const int start = blockIdx.x * R;
  if (start >= n) return;
  const int rows = min(R, n - start), C = p.C(), cq = p.hq * p.dk, m = p.taps - 1;
  const bool on = 8 * (int)threadIdx.x < C;
  const int c = on ? 8 * threadIdx.x : 0;
  const bool is_k = c >= cq;
  const T* base = p.x + (int64_t)(q0 + start) * p.ld;
  float* ring = m > 0 ? p.state + (int64_t)p.slots[s] * p.slot_stride : nullptr;
  const int half = p.rot / 2, pair = c % p.dk / 2;
  const bool turns = on && pair < half;
  const int* table = p.tables + (int64_t)s * p.max_blocks;
  const int slot_len = p.hkv * (p.dk + p.dv);
  Raw<T, 8> x;
  x.load(base + c);
  // [k]: k + 1 back for hist, k back for w
  float w[M + 1][8], hist[M + 1][8], nw[8];
  if (start > 0) {
    Raw<T, 8> h[M + 1];
#pragma unroll
    for (int k = 0; k < M; ++k) h[k].load(base - (int64_t)min(k + 1, start) * p.ld + c);
#pragma unroll
    for (int k = 0; k < M; ++k)
#pragma unroll
      for (int i = 0; i < 8; ++i) hist[k][i] = h[k][i];
  } else {
#pragma unroll
    for (int k = 0; k < M; ++k) {
#pragma unroll
      for (int i = 0; i < 8; ++i) hist[k][i] = 0.f;
      if (k < m && k < seen) Vec8<float>::load(ring + (int64_t)((seen - 1 - k) % p.taps) * C + c, hist[k]);
    }
  }
#pragma unroll
  for (int k = 0; k <= M; ++k) {  // (rows of weights past the taps count nothing)
#pragma unroll
    for (int i = 0; i < 8; ++i) w[k][i] = k == 0 ? 1.f : 0.f;
    if (p.cw != nullptr && k <= m) Vec8<float>::load(p.cw + (m - k) * C + c, w[k]);
  }
#pragma unroll
  for (int i = 0; i < 8; ++i) nw[i] = 1.f;
  if (p.qn != nullptr) Vec8<float>::load(is_k ? p.kn + c - cq : p.qn + c, nw);
  const float inv_q = 1.f / (float)p.width_q, inv_k = 1.f / (float)p.width_k;
  for (int r = 0; r < rows; ++r) {
    const int64_t row = q0 + start + r;
    const int pos = seen + start + r;
    T* at = p.cache + ((int64_t)table[pos / p.block_size] * p.block_size + pos % p.block_size) * slot_len;
    float u[8], cs[4], sn[4], ss = 0.f;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      cs[j] = 1.f;
      sn[j] = 0.f;
    }
    if (turns) {
      const float* cp = p.cos_t + (int64_t)pos * half + pair;
      const float* sp = p.sin_t + (int64_t)pos * half + pair;
      if ((half & 3) == 0) {
        VecN<float, 4>::load(cp, cs);
        VecN<float, 4>::load(sp, sn);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (pair + j < half) {
            cs[j] = cp[j];
            sn[j] = sp[j];
          }
      }
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const float now = x[i];
      u[i] = w[0][i] * now;
#pragma unroll
      for (int k = 0; k < M; ++k) u[i] += w[k + 1][i] * hist[k][i];
      ss += u[i] * u[i];
#pragma unroll
      for (int k = M - 1; k > 0; --k) hist[k][i] = hist[k - 1][i];
      hist[0][i] = now;
    }
    if (r + 1 < rows) x.load(base + (int64_t)(r + 1) * p.ld + c);
    float f = 1.f;
    if (p.qn != nullptr) {
      float sum = 0.f;
      if (p.sums_in == nullptr) {
        const float a = wave_sum(on && !is_k ? ss : 0.f), b = wave_sum(on && is_k ? ss : 0.f);
        if ((threadIdx.x & 63) == 0) {
          red[r & 1][0][threadIdx.x >> 6] = a;
          red[r & 1][1][threadIdx.x >> 6] = b;
        }
        __syncthreads();
#pragma unroll
        for (int j = 0; j < NW; ++j) sum += red[r & 1][is_k][j];
        if (p.sums_out != nullptr) {
          if (on && (c == 0 || c == cq)) p.sums_out[2 * row + is_k] = sum;
          continue;
        }
      } else {
        sum = p.sums_in[2 * row + is_k];
      }
      f = rsqrtf(sum * (is_k ? inv_k : inv_q) + p.eps);
    }
    if (!p.shared)
      for (int e = 8 * threadIdx.x; e < p.hkv * p.dv; e += 8 * NT) {
        float v[8];
        Vec8<T>::load(p.x + row * p.ld + C + e, v);
        Vec8<T>::store(at + p.hkv * p.dk + e, v);
      }
    if (!on) continue;
    if (is_k && p.shared) Vec8<T>::store(at + p.hkv * p.dk + c - cq, u);
#pragma unroll
    for (int i = 0; i < 8; ++i) u[i] *= f * nw[i];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const float a = u[2 * j], b = u[2 * j + 1];
      u[2 * j] = a * cs[j] - b * sn[j];
      u[2 * j + 1] = b * cs[j] + a * sn[j];
    }
    Vec8<T>::store(is_k ? at + c - cq : p.q + row * p.ldq + c, u);
  }
  if (blockIdx.x == 0 && on && m > 0 && p.sums_out == nullptr)
    for (int i0 = max(n - m, 0); i0 < n; ++i0) {
      float v[8];
      VecN<T, 8>::load(base + (int64_t)i0 * p.ld + c, v);
      Vec8<float>::store(ring + (int64_t)((seen + i0) % p.taps) * C + c, v);
    }
}

// any sizes: the row in LDS
template <typename T>
__global__ __launch_bounds__(256) void head_prep_kernel(PrepParams<T> p) {
  extern __shared__ float sm[];
  __shared__ float red[2][4];
  const Token<T> k = token_of(p, blockIdx.x);
  const int C = p.C(), cq = p.hq * p.dk;
  float sq = 0.f, sk = 0.f;
  for (int c = threadIdx.x; c < C; c += 256) {
    float u[1];
    convolve<T, 1>(p, k, c, u);
    sm[c] = u[0];
    if (c < cq) sq += u[0] * u[0]; else sk += u[0] * u[0];
  }
  two_sums<256>(sq, sk, red);  // (also the barrier in front of the reads of sm)
  if (p.sums_out != nullptr) {
    if (threadIdx.x < 2) p.sums_out[2 * (int64_t)k.row + threadIdx.x] = threadIdx.x == 0 ? sq : sk;
    return;
  }
  float rq, rk;
  norm_factors(p, k, sq, sk, rq, rk);
  const int half = p.rot / 2;
  for (int c = threadIdx.x; c < C; c += 256) {
    const bool is_k = c >= cq;
    const float r = is_k ? rk : rq;
    const float* n = p.qn == nullptr ? nullptr : (is_k ? p.kn - cq : p.qn);
    if (is_k && p.shared) k.slot[p.hkv * p.dk + c - cq] = from_f<T>(sm[c]);
    float v = sm[c] * r * (n != nullptr ? n[c] : 1.f);
    const int e = c % p.dk;
    if (e < p.rot) {
      const int o = e & 1 ? c - 1 : c + 1;
      const float u = sm[o] * r * (n != nullptr ? n[o] : 1.f);
      const float cs = p.cos_t[(int64_t)k.pos * half + e / 2], sn = p.sin_t[(int64_t)k.pos * half + e / 2];
      v = e & 1 ? v * cs + u * sn : v * cs - u * sn;
    }
    if (is_k) k.slot[c - cq] = from_f<T>(v);
    else p.q[(int64_t)k.row * p.ldq + c] = from_f<T>(v);
  }
  if (!p.shared)
    for (int c = threadIdx.x; c < p.hkv * p.dv; c += 256) k.slot[p.hkv * p.dk + c] = p.x[(int64_t)k.row * p.ld + C + c];
}

// last inputs of portions of two and more tokens
template <typename T>
__global__ __launch_bounds__(256) void head_tail_kernel(PrepParams<T> p) {
  const int s = blockIdx.y, q0 = p.seq_meta[3 * s], n = p.seq_meta[3 * s + 1], seen = p.seq_meta[3 * s + 2];
  const int C = p.C(), c = blockIdx.x * 256 + threadIdx.x;
  if (n < 2 || c >= C) return;
  float* ring = p.state + (int64_t)p.slots[s] * p.slot_stride + c;
  for (int i = max(n - (p.taps - 1), 0); i < n; ++i)
    ring[(int64_t)((seen + i) % p.taps) * C] = to_f(p.x[(int64_t)(q0 + i) * p.ld + c]);
}

template <typename T>
int launch_prep(const PrepParams<T>& p, int n_seqs, int max_new, hipStream_t st) {
  const int C = p.C();
  const bool v8 = p.dk % 8 == 0 && p.dv % 8 == 0 && p.ld % 8 == 0 && p.ldq % 8 == 0 && p.slot_stride % 4 == 0 &&
                  (uintptr_t)p.x % 16 == 0 && (uintptr_t)p.q % 16 == 0 && (uintptr_t)p.cache % 16 == 0 &&
                  (uintptr_t)p.state % 16 == 0;
  if (v8 && max_new > 1 && (C <= 4096 ? p.taps <= 8 : C <= 8192 && p.taps <= 4)) {
    // (a longer run reads its weights and last inputs less often, if there are enough of them)
    const int R = p.taps > 4 || (C > 2048 && (int64_t)max_new * n_seqs >= 4096) ? 8 : 4;
    const dim3 grid((max_new + R - 1) / R, n_seqs);
#define HDS_HR(NT, MM, OO) hipLaunchKernelGGL((head_prep_run_kernel<T, NT, MM, OO>), grid, dim3(NT), 0, st, p, R)
#define HDS_HRM(NT) { if (p.taps <= 4) HDS_HR(NT, 3, 4); else HDS_HR(NT, 7, 2); }
    if (C <= 2048) HDS_HRM(256) else if (C <= 4096) HDS_HRM(512) else HDS_HR(1024, 3, 4);
#undef HDS_HRM
#undef HDS_HR
    return hipGetLastError();
  }
#define HDS_HP(NC, NT) hipLaunchKernelGGL((head_prep8_kernel<T, NC, NT>), dim3(p.n_tok), dim3(NT), 0, st, p)
  if (v8 && C <= 16384) {
    if (p.n_tok <= 64 && C > 2048) {  // few rows: many threads on each
      if (C <= 8192) HDS_HP(1, 1024); else HDS_HP(2, 1024);
    } else if (C <= 2048) {
      HDS_HP(1, 256);
    } else if (C <= 4096) {
      HDS_HP(1, 512);
    } else if (C <= 8192) {
      HDS_HP(2, 512);
    } else {
      HDS_HP(4, 512);
    }
  } else {
    if (C > 15 * 1024) return hipErrorInvalidValue;
    hipLaunchKernelGGL(head_prep_kernel<T>, dim3(p.n_tok), dim3(256), C * sizeof(float), st, p);
  }
#undef HDS_HP
  if (const hipError_t e = hipGetLastError()) return e;
  if (p.taps > 1 && max_new > 1 && p.sums_out == nullptr) {
    hipLaunchKernelGGL(head_tail_kernel<T>, dim3((C + 255) / 256, n_seqs), dim3(256), 0, st, p);
    return hipGetLastError();
  }
  return 0;
}

}  // namespace

// See PrepParams. shared: dv == dk and x has no value columns. cw null: taps 1. sums_out: only the sums are written (the ring
// entries of lone tokens too, which the second call writes again); sums_in: with the norms' total sums.
HDS_EXPORT int hds_head_prep(int dtype, const void* x, int64_t ld, int hq, int hkv, int dk, int dv, int taps, int rot,
                             int shared, const float* cw, const float* qn, const float* kn, const float* cos_t,
                             const float* sin_t, void* q, int64_t ldq, void* cache, const int* tables, int max_blocks,
                             int block_size, const int* tok_seq, const int* tok_pos, const int* seq_meta, float* state,
                             int64_t slot_stride, const int* slots, float* sums_out, const float* sums_in, int width_q,
                             int width_k, float eps, int n_tok, int n_seqs, int max_new, hipStream_t st) {
  if (n_tok <= 0) return 0;
  if (hq < 1 || hkv < 1 || hq % hkv || dk < 1 || dv < 1 || taps < 1 || (cw == nullptr && taps != 1) || rot < 0 || rot % 2 ||
      rot > dk || (shared && dv != dk) || ld < (int64_t)(hq + hkv) * dk + (shared ? 0 : (int64_t)hkv * dv) ||
      ldq < (int64_t)hq * dk || (rot > 0 && (cos_t == nullptr || sin_t == nullptr)) || (qn == nullptr) != (kn == nullptr) ||
      (taps > 1 && (state == nullptr || slots == nullptr || slot_stride < (int64_t)taps * (hq + hkv) * dk)) || width_q < 1 || width_k < 1 ||
      n_seqs < 1 || n_seqs > 65535 || (sums_out != nullptr && (sums_in != nullptr || qn == nullptr)))
    return hipErrorInvalidValue;
#define HDS_PP(TT)                                                                                                     \
  return launch_prep(PrepParams<TT>{(const TT*)x, ld, hq, hkv, dk, dv, taps, rot, shared, cw, qn, kn, cos_t, sin_t,   \
                                    (TT*)q, ldq, (TT*)cache, tables, max_blocks, block_size, tok_seq, tok_pos,        \
                                    seq_meta, state, slot_stride, slots, sums_out, sums_in, width_q, width_k, eps,    \
                                    n_tok}, n_seqs, max_new, st)
  if (dtype == kBF16) HDS_PP(bf16);
  if (dtype == kF32) HDS_PP(float);
#undef HDS_PP
  return hipErrorInvalidValue;
}
