// Matrix memories of a recurrent mixer over ragged batches: linear attention with a decay and, optionally, exponential
// gates under a running maximum. A head h carries a 32-bit state S [dk, dv]; per token, with log decay f and log input
// gate i,
//
//   m' = max(f + m, i),   S' = e^(f + m - m') S + e^(i - m') k v^T,   o = S'^T q * dk^(-1/2)
//
// Two kinds:
//   fixed:  f is a constant per head, i = 0 (so m stays 0): retention.
//   gated:  i = cap tanh((zi + bi) / cap), f = log sigmoid(cap tanh((zf + bf) / cap)); n' is S' with k alone, and
//           o <- o / (max(|n' . q dk^(-1/2)|, e^(-m')) + 1e-6). m starts at 0.
// q and k may be rotated (neighbouring pairs of the first `rot` dimensions). Then
//
//   out = o / sqrt(mean(o^2) + eps) * w * act(gate)       (w optional, act: sigmoid or silu)
//
// One projection row holds q [H dk] | k [H dk] | v [H dv] | gate [H dv], and zi [H] | zf [H] of the gated kind. A sequence's
// slot holds, head by head, S and then n [dk] of the gated kind, and behind all heads m [H]. A sequence whose `seen` is 0
// starts from zero whatever the slot holds.
//
// Single tokens run one kernel, a workgroup per (sequence, head): memory_step. Portions are scanned token by token
// (memory_gates, memory_scan, memory_out: short portions, 32-bit engines, any sizes) or by chunks of 64 on the matrix cores:
//   memory_chunk_sum   every chunk's own sum of e^(..) k v^T, all chunks at once
//   memory_chunk_walk  elementwise over the chunks: leaves the state in front of every chunk where the sum was
//   memory_chunk_out   all chunks at once: what the state in front gives, what the chunk's own tokens give, norm and gate
// The state does not feed back into what is written, so only the walk is sequential, and it moves memory only.
#include "hds_common.h"

namespace {
using namespace hds;

constexpr float kFloorEps = 1e-6f;
constexpr int kSigmoidGate = 0;

__device__ __forceinline__ float sigmoid_f(float x) {
  const float e = expf(-fabsf(x)), r = 1.f / (1.f + e);
  return x >= 0.f ? r : e * r;
}
__device__ __forceinline__ float log_sigmoid_f(float x) { return fminf(x, 0.f) - log1pf(expf(-fabsf(x))); }
// of output gates (rounded to T)
template <typename T>
__device__ __forceinline__ float gate_act(float x, int act) {
  float s;
  if constexpr (sizeof(T) == 2) s = __builtin_amdgcn_rcpf(1.f + __expf(-x));
  else s = sigmoid_f(x);
  return act == kSigmoidGate ? s : x * s;
}

struct MemoryDims {
  int H, dk, dv, rot, gated;
  int64_t ld;  // row stride of the projection
  __device__ __host__ __forceinline__ int k0() const { return H * dk; }
  __device__ __host__ __forceinline__ int v0() const { return 2 * H * dk; }
  __device__ __host__ __forceinline__ int g0() const { return 2 * H * dk + H * dv; }
  __device__ __host__ __forceinline__ int i0() const { return 2 * H * (dk + dv); }
  __device__ __host__ __forceinline__ int width() const { return i0() + (gated ? 2 * H : 0); }
  __device__ __host__ __forceinline__ int used() const { return dk * dv + (gated ? dk : 0); }  // floats of a head
  __device__ __host__ __forceinline__ int head() const { return (used() + 3) & ~3; }
  __device__ __host__ __forceinline__ int64_t states() const { return (int64_t)H * head() + (gated ? H : 0); }
};

template <typename T>
struct MemoryParams {
  MemoryDims d;
  const T* proj;         // [tokens, d.ld]
  const float* log_decay;  // [H], fixed kind
  const float* bi;       // [H], gated kind
  const float* bf;
  float cap;
  const float* cos_t;    // [positions, rot / 2]
  const float* sin_t;
  const float* norm;     // [H dv] or null
  int act;
  float* state;          // [slots] x slot_stride
  int64_t slot_stride;
  const int* slots;
  const int* seq_meta;   // [sequences][3] = {first row, new tokens, seen}
  const int* seqs;       // the sequences this launch works on; null: 0, 1, ..
  float* coef;           // [tokens, H, 4]: factor of S, factor of k v^T, e^(-m), denominator
  float* o;              // [tokens, H, dv] read-outs
  T* out;                // [tokens, ldo]
  int64_t ldo;
  float eps;
};

struct Seq {
  int q0, n, seen, slot;
};
template <typename T>
__device__ __forceinline__ Seq seq_of(const MemoryParams<T>& p, int i) {
  const int s = p.seqs != nullptr ? p.seqs[i] : i;
  return {p.seq_meta[3 * s], p.seq_meta[3 * s + 1], p.seq_meta[3 * s + 2], p.slots[s]};
}
template <typename T>
__device__ __forceinline__ float* head_state(const MemoryParams<T>& p, const Seq& s, int h) {
  return p.state + (int64_t)s.slot * p.slot_stride + (int64_t)h * p.d.head();
}
template <typename T>
__device__ __forceinline__ float* head_max(const MemoryParams<T>& p, const Seq& s, int h) {
  return p.state + (int64_t)s.slot * p.slot_stride + (int64_t)p.d.H * p.d.head() + h;
}

// log decay and log input gate of row t
template <typename T>
__device__ __forceinline__ void log_gates(const MemoryParams<T>& p, int64_t t, int h, float& f, float& i) {
  if (!p.d.gated) {
    f = p.log_decay[h];
    i = 0.f;
    return;
  }
  const T* z = p.proj + t * p.d.ld + p.d.i0() + h;
  i = p.cap * tanhf((to_f(z[0]) + p.bi[h]) / p.cap);
  f = log_sigmoid_f(p.cap * tanhf((to_f(z[p.d.H]) + p.bf[h]) / p.cap));
}

// element e of a head's q or k (x: its start) at position pos, rotated
template <typename T>
__device__ __forceinline__ float rotated(const MemoryParams<T>& p, const T* x, int e, int pos) {
  const float v = to_f(x[e]);
  if (e >= p.d.rot) return v;
  const int64_t a = (int64_t)pos * (p.d.rot / 2) + (e >> 1);
  const float u = to_f(x[e ^ 1]), c = p.cos_t[a], s = p.sin_t[a];
  return e & 1 ? v * c + u * s : v * c - u * s;
}

// cosines and sines of the four pairs from element e (a multiple of 8) on, at position pos
struct Turn {
  float c[4], s[4];
};
template <typename T>
__device__ __forceinline__ Turn turn_of(const MemoryParams<T>& p, int e, int pos) {
  const int half = p.d.rot / 2;
  Turn t;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    t.c[j] = 1.f;
    t.s[j] = 0.f;
  }
  if (e >= p.d.rot) return t;
  const float* cp = p.cos_t + (int64_t)pos * half + e / 2;
  const float* sp = p.sin_t + (int64_t)pos * half + e / 2;
  if ((half & 3) == 0) {
    VecN<float, 4>::load(cp, t.c);
    VecN<float, 4>::load(sp, t.s);
  } else {
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (e / 2 + j < half) {
        t.c[j] = cp[j];
        t.s[j] = sp[j];
      }
  }
  return t;
}
// the elements as numbers, turned
template <bool TURNS>
__device__ __forceinline__ void turned(const bf16x8& x, const Turn& t, float (&v)[8]) {
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const float a = (float)x[2 * j], b = (float)x[2 * j + 1];
    v[2 * j] = TURNS ? a * t.c[j] - b * t.s[j] : a;
    v[2 * j + 1] = TURNS ? b * t.c[j] + a * t.s[j] : b;
  }
}

// ---------------------------------------------------------------------------------------------------------------
// scan, token by token
// ---------------------------------------------------------------------------------------------------------------
// What the tokens before and at lane l of a run of up to 64 do together: G, the sum of the log decays, and P, the largest
// i - G. The maximum after token l is G + max(m in front, P).
__device__ __forceinline__ void run_sums(float f, float i, float& G, float& P) {
  const int lane = threadIdx.x & 63;
  G = f;
#pragma unroll
  for (int o = 1; o < 64; o <<= 1) {
    const float v = __shfl_up(G, o, 64);
    if (lane >= o) G += v;
  }
  P = i - G;
#pragma unroll
  for (int o = 1; o < 64; o <<= 1) {
    const float v = __shfl_up(P, o, 64);
    if (lane >= o) P = fmaxf(P, v);
  }
}

// gated kind: factors of every token, one wave per (head, sequence)
template <typename T>
__global__ __launch_bounds__(64) void memory_gates_kernel(MemoryParams<T> p) {
  const Seq s = seq_of(p, blockIdx.y);
  const int h = blockIdx.x, lane = threadIdx.x;
  if (s.n <= 0) return;
  float* mp = head_max(p, s, h);
  float m = s.seen > 0 ? *mp : 0.f;
  float f = 0.f, i = 0.f, fn, in;
  auto fetch = [&](int t0, float& a, float& b) {
    a = 0.f;
    b = -INFINITY;
    if (t0 + lane < s.n) log_gates(p, s.q0 + t0 + lane, h, a, b);
  };
  fetch(0, fn, in);
  for (int t0 = 0; t0 < s.n; t0 += 64) {
    f = fn;
    i = in;
    if (t0 + 64 < s.n) fetch(t0 + 64, fn, in);
    float G, P;
    run_sums(f, i, G, P);
    const float now = G + fmaxf(m, P);
    float before = __shfl_up(now, 1, 64);
    if (lane == 0) before = m;
    if (t0 + lane < s.n) {
      float* c = p.coef + 4 * ((int64_t)(s.q0 + t0 + lane) * p.d.H + h);
      c[0] = expf(f + before - now);
      c[1] = expf(i - now);
      c[2] = expf(-now);
    }
    m = __shfl(now, min(63, s.n - 1 - t0), 64);
  }
  if (lane == 0) *mp = m;
}

constexpr int kScanTok = 8;  // tokens staged at a time

// a workgroup per 64 columns of one head's state, R rows of it in each wave's registers
template <typename T, int R>
__global__ __launch_bounds__(256) void memory_scan_kernel(MemoryParams<T> p) {
  __shared__ float sq[kScanTok][4 * R], sk[kScanTok][4 * R];
  __shared__ float part[kScanTok][4][64], pn[kScanTok][4];
  __shared__ float sc[kScanTok][3];
  const Seq s = seq_of(p, blockIdx.z);
  if (s.n <= 0) return;
  const MemoryDims& d = p.d;
  const int h = blockIdx.y, lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int col = blockIdx.x * 64 + lane, dk = d.dk, dv = d.dv;
  const bool ok = col < dv, norms = d.gated && blockIdx.x == 0;  // n: kept by the first columns' workgroup
  const int cc = ok ? col : dv - 1;
  float* st = head_state(p, s, h);
  const float scale = 1.f / sqrtf((float)dk);
  float S[R], n[2];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int row = w * R + r;
    S[r] = s.seen > 0 && row < dk ? st[(int64_t)row * dv + cc] : 0.f;
  }
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int e = threadIdx.x + 256 * j;
    n[j] = norms && s.seen > 0 && e < dk ? st[(int64_t)dk * dv + e] : 0.f;
  }
  const float fixed = d.gated ? 0.f : expf(p.log_decay[h]);
  for (int t0 = 0; t0 < s.n; t0 += kScanTok) {
    const int nt = min(kScanTok, s.n - t0);
    for (int x = threadIdx.x; x < nt * 4 * R; x += 256) {
      const int i = x / (4 * R), e = x - i * 4 * R;
      const T* row = p.proj + (int64_t)(s.q0 + t0 + i) * d.ld + h * dk;
      const int pos = s.seen + t0 + i;
      sq[i][e] = e < dk ? rotated(p, row, e, pos) * scale : 0.f;
      sk[i][e] = e < dk ? rotated(p, row + d.k0(), e, pos) : 0.f;
    }
    if ((int)threadIdx.x < nt * 3) {
      const int i = threadIdx.x / 3, c = threadIdx.x % 3;
      sc[i][c] = d.gated ? p.coef[4 * ((int64_t)(s.q0 + t0 + i) * d.H + h) + c] : (c == 0 ? fixed : 1.f);
    }
    __syncthreads();
    float vn = to_f(p.proj[(int64_t)(s.q0 + t0) * d.ld + d.v0() + h * dv + cc]);
    for (int i = 0; i < nt; ++i) {
      const float v = vn * sc[i][1], keep = sc[i][0];
      if (i + 1 < nt) vn = to_f(p.proj[(int64_t)(s.q0 + t0 + i + 1) * d.ld + d.v0() + h * dv + cc]);
      float qs = 0.f;
#pragma unroll
      for (int r = 0; r < R; ++r) {
        S[r] = keep * S[r] + sk[i][w * R + r] * v;
        qs += S[r] * sq[i][w * R + r];
      }
      part[i][w][lane] = qs;
      if (norms) {
        float nq = 0.f;
#pragma unroll
        for (int j = 0; j < 2; ++j) {
          const int e = threadIdx.x + 256 * j;
          if (e < dk) {
            n[j] = keep * n[j] + sc[i][1] * sk[i][e];
            nq += n[j] * sq[i][e];
          }
        }
        nq = wave_sum(nq);
        if (lane == 0) pn[i][w] = nq;
      }
    }
    __syncthreads();
    for (int i = w; i < nt; i += 4) {
      const int64_t at = (int64_t)(s.q0 + t0 + i) * d.H + h;
      if (ok) p.o[at * dv + col] = part[i][0][lane] + part[i][1][lane] + part[i][2][lane] + part[i][3][lane];
      if (norms && lane == 0)
        p.coef[4 * at + 3] = fmaxf(fabsf(pn[i][0] + pn[i][1] + pn[i][2] + pn[i][3]), sc[i][2]) + kFloorEps;
    }
    __syncthreads();
  }
  if (ok)
#pragma unroll
    for (int r = 0; r < R; ++r)
      if (w * R + r < dk) st[(int64_t)(w * R + r) * dv + col] = S[r];
  if (norms)
#pragma unroll
    for (int j = 0; j < 2; ++j)
      if ((int)threadIdx.x + 256 * j < dk) st[(int64_t)dk * dv + threadIdx.x + 256 * j] = n[j];
}

// denominator, norm and gate: one wave per (token, head)
template <typename T>
__global__ __launch_bounds__(256) void memory_out_kernel(MemoryParams<T> p) {
  const Seq s = seq_of(p, blockIdx.y);
  const int lane = threadIdx.x & 63, dv = p.d.dv;
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  const int t = (int)(item / p.d.H), h = (int)(item % p.d.H);
  if (t >= s.n) return;
  const int64_t row = s.q0 + t, at = row * p.d.H + h;
  const float inv = p.d.gated ? 1.f / p.coef[4 * at + 3] : 1.f;
  const float* o = p.o + at * dv;
  const T* g = p.proj + row * p.d.ld + p.d.g0() + h * dv;
  float ss = 0.f;
  for (int e = lane; e < dv; e += 64) ss += (o[e] * inv) * (o[e] * inv);
  const float rs = inv / sqrtf(wave_sum(ss) / (float)dv + p.eps);
  for (int e = lane; e < dv; e += 64)
    p.out[row * p.ldo + h * dv + e] =
        from_f<T>(o[e] * rs * (p.norm != nullptr ? p.norm[h * dv + e] : 1.f) * gate_act<T>(to_f(g[e]), p.act));
}

// ---------------------------------------------------------------------------------------------------------------
// one token per sequence: a workgroup per (head, sequence)
// ---------------------------------------------------------------------------------------------------------------
// A thread keeps 4 columns of RPT rows of S; one pass reads, advances, reads out and stores them.
template <typename T, int RPT, int NT>
__global__ __launch_bounds__(NT, NT < 1024 ? 1 : (RPT <= 4 ? 8 : 4)) void memory_step_kernel(MemoryParams<T> p) {
  constexpr int NW = NT / 64;
  extern __shared__ float sm[];
  __shared__ float red[2][NW];
  const MemoryDims& d = p.d;
  const int dk = d.dk, dv = d.dv, cq = dv / 4;
  const int RG = NT / cq;                     // row groups
  const bool fold = (cq & (cq - 1)) == 0 && cq <= 64;  // the row groups of a wave reduce by lane exchange
  const int P = fold ? NW : RG;
  float* part = sm;                           // [P][dv]
  float* sq = part + P * dv;                  // [dk]
  float* sk = sq + dk;                        // [dk]
  const int h = blockIdx.x;
  const Seq s = seq_of(p, blockIdx.y);
  if (s.n != 1) return;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, tid = threadIdx.x;
  const int c4 = tid % cq, rg = tid / cq;
  const bool act = rg < RG;
  float* st = head_state(p, s, h);
  float* Sp = st + 4 * c4;
  const T* row = p.proj + (int64_t)s.q0 * d.ld;
  const float scale = 1.f / sqrtf((float)dk);
  // q, k and the gates first, then S, in the order of their use
  float qk = 0.f;
  if (tid < 2 * dk) {
    const bool is_k = tid >= dk;
    qk = rotated(p, row + (is_k ? d.k0() : 0) + h * dk, is_k ? tid - dk : tid, s.seen) * (is_k ? 1.f : scale);
  }
  float f, i;
  log_gates(p, s.q0, h, f, i);
  float* mp = d.gated ? head_max(p, s, h) : nullptr;
  const float m0 = d.gated && s.seen > 0 ? *mp : 0.f;
  f32x4 S[RPT];
#pragma unroll
  for (int r = 0; r < RPT; ++r) {
    S[r] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int e = rg + r * RG;
    if (act && s.seen > 0 && e < dk) S[r] = *reinterpret_cast<const f32x4*>(Sp + (int64_t)e * dv);
  }
  float v[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) v[j] = to_f(row[d.v0() + h * dv + 4 * c4 + j]);
  const int o_first = min(tid, dv - 1);
  const float og = to_f(row[d.g0() + h * dv + o_first]), nw = p.norm != nullptr ? p.norm[h * dv + o_first] : 1.f;
  float n0 = 0.f;
  if (d.gated && tid < dk && s.seen > 0) n0 = st[(int64_t)dk * dv + tid];
  const float m = fmaxf(f + m0, i), keep = expf(f + m0 - m), add = expf(i - m);
  if (tid < 2 * dk) sq[tid] = qk;
  for (int e = NT + tid; e < 2 * dk; e += NT)
    sq[e] = rotated(p, row + (e >= dk ? d.k0() : 0) + h * dk, e >= dk ? e - dk : e, s.seen) * (e >= dk ? 1.f : scale);
  __syncthreads();
  f32x4 qs = {0.f, 0.f, 0.f, 0.f};
  const f32x4 av = {add * v[0], add * v[1], add * v[2], add * v[3]};
#pragma unroll
  for (int r = 0; r < RPT; ++r) {
    const int e = rg + r * RG;
    if (act && e < dk) {
      S[r] = keep * S[r] + sk[e] * av;
      qs += S[r] * sq[e];
      *reinterpret_cast<f32x4*>(Sp + (int64_t)e * dv) = S[r];
    }
  }
  if (d.gated) {
    float nq = 0.f;
    for (int e = tid; e < dk; e += NT) {
      const float old = e == tid ? n0 : (s.seen > 0 ? st[(int64_t)dk * dv + e] : 0.f);
      const float nn = keep * old + add * sk[e];
      st[(int64_t)dk * dv + e] = nn;
      nq += nn * sq[e];
    }
    nq = wave_sum(nq);
    if (lane == 0) red[0][w] = nq;
  }
  if (fold) {
    for (int off = cq; off < 64; off <<= 1)
#pragma unroll
      for (int j = 0; j < 4; ++j) qs[j] += __shfl_xor(qs[j], off, 64);
    if (lane < cq) *reinterpret_cast<f32x4*>(part + w * dv + 4 * c4) = qs;
  } else if (act) {
    *reinterpret_cast<f32x4*>(part + rg * dv + 4 * c4) = qs;
  }
  __syncthreads();
  float inv = 1.f;
  if (d.gated) {
    float nq = 0.f;
#pragma unroll
    for (int x = 0; x < NW; ++x) nq += red[0][x];
    inv = 1.f / (fmaxf(fabsf(nq), expf(-m)) + kFloorEps);
    if (tid == 0) *mp = m;
  }
  // every thread's own columns stay in registers: dv <= 1024 <= 4 NT
  float o[4], ss = 0.f;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int c = tid + j * NT;
    o[j] = 0.f;
    if (c < dv) {
#pragma unroll 8
      for (int x = 0; x < P; ++x) o[j] += part[x * dv + c];
      o[j] *= inv;
      ss += o[j] * o[j];
    }
  }
  ss = wave_sum(ss);
  if (lane == 0) red[1][w] = ss;
  __syncthreads();
  ss = 0.f;
#pragma unroll
  for (int x = 0; x < NW; ++x) ss += red[1][x];
  const float rs = 1.f / sqrtf(ss / (float)dv + p.eps);
  T* op = p.out + (int64_t)s.q0 * p.ldo + h * dv;
  if (tid < dv) op[tid] = from_f<T>(o[0] * rs * nw * gate_act<T>(og, p.act));
#pragma unroll
  for (int j = 1; j < 4; ++j) {
    const int c = tid + j * NT;
    if (c < dv)
      op[c] = from_f<T>(o[j] * rs * (p.norm != nullptr ? p.norm[h * dv + c] : 1.f) *
                        gate_act<T>(to_f(row[d.g0() + h * dv + c]), p.act));
  }
}

// ---------------------------------------------------------------------------------------------------------------
// scan by chunks of 64 tokens
// ---------------------------------------------------------------------------------------------------------------
// With G and P as in run_sums over a chunk's tokens, S, n and m in front of the chunk, F = G_last, and
// m_t = G_t + max(m, P_t):
//
//   sum   = sum_j e^(F - G_j + i_j - b) k_j v_j^T,             b = F + P_last  (F = b = 0 of no tokens)
//   S_out = e^(F + m - m_out) S + e^(b - m_out) sum,           m_out = max(F + m, b)
//   o_t   = e^(G_t + m - m_t) S^T q_t + sum_(j <= t) A_tj v_j, A_tj = e^(G_t - G_j + i_j - m_t) q_t . k_j
//
// and likewise n with v = 1. All of it is 32-bit: v is bfloat16, and so are q and k where they are not rotated; everything
// else enters its products as a sum of three bfloat16 numbers (24 bits), of whose products those above 2^-24 are kept.
constexpr int kChunk = 64;
constexpr int kPadRow = 8;  // bfloat16 numbers behind a row in LDS

// Scratch memory of a chunk and head: sum, then state in front [head floats] | F, b, m in front, -. The chunks of sequence i
// start at q0 / 64 + i (they do not overlap).
struct ChunkWs {
  float* base;
  int64_t floats;  // per chunk and head
  __device__ __forceinline__ float* at(const Seq& s, int i, int chunk, int h, int H) const {
    return base + ((int64_t)(s.q0 / kChunk + i + chunk) * H + h) * floats;
  }
};

__device__ __forceinline__ f32x4 mfma_bf16(const bf16x8& a, const bf16x8& b, const f32x4& c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

// x as a sum of N bfloat16 numbers
template <int N>
__device__ __forceinline__ void split8(const float (&x)[8], bf16x8 (&out)[N]) {
  float r[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) r[i] = x[i];
#pragma unroll
  for (int k = 0; k < N; ++k)
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const bf16 v = (bf16)r[i];
      out[k][i] = v;
      r[i] -= (float)v;
    }
}

// transposed LDS read: lane (g = lane / 16, c = lane % 16) gets rows 4 g .. 4 g + 3 of column c of a block of 16 columns;
// `tile` is the block's first row and column
__device__ __forceinline__ bf16x4 read_tr(const bf16* tile, int ld) {
  const int lane = threadIdx.x & 63, l15 = lane & 15, g = lane >> 4;
  const bf16* a = tile + (4 * g + (l15 >> 2)) * ld + 4 * (l15 & 3);
  return __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) bf16x4*)(a));
}
// 32 tokens of 16 columns as a matrix operand: lane group g holds tokens 4 g .. + 3 of the first and of the second 16
__device__ __forceinline__ bf16x8 read_tokens(const bf16* tile, int ld) {
  return __builtin_shufflevector(read_tr(tile, ld), read_tr(tile + 16 * ld, ld), 0, 1, 2, 3, 4, 5, 6, 7);
}

// KT: 16-row tiles of the state a wave has (dk <= 64 KT). Everything a thread reads is requested at once.
// LPV lanes a token of v (dv <= 8 LPV).
template <int KT, bool TURNS, int LPV>
__global__ __launch_bounds__(256) void memory_chunk_sum_kernel(MemoryParams<bf16> p, ChunkWs ws) {
  extern __shared__ __attribute__((aligned(16))) bf16 lds[];  // k e^(..) in three planes [64][ldk], v [64][ldv]
  __shared__ float sw[kChunk];
  const Seq s = seq_of(p, blockIdx.z);
  const int chunk = blockIdx.x, h = blockIdx.y, left = s.n - chunk * kChunk;
  if (left <= 0) return;
  const MemoryDims& d = p.d;
  const int dk = d.dk, dv = d.dv, kp = (dk + 15) / 16 * 16, vp = (dv + 15) / 16 * 16;
  const int ldk = kp + kPadRow, ldv = vp + kPadRow;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, l15 = lane & 15, g = lane >> 4;
  const int64_t t0 = s.q0 + chunk * kChunk;
  const int pos0 = s.seen + chunk * kChunk;
  float* out = ws.at(s, blockIdx.z, chunk, h, d.H);
  bf16* sv = lds + 3 * kChunk * ldk;
  // missing tokens have weight zero and repeat the last one
  constexpr int LPK = 8 * KT, NK = 64 * LPK / 256, NV = 64 * LPV / 256;
  const int ke = 8 * (threadIdx.x % LPK), ve = 8 * (threadIdx.x % LPV);
  bf16x8 kx[NK], vx[NV];
  Turn turn[NK];
#pragma unroll
  for (int y = 0; y < NK; ++y) {
    const int tt = min((int)threadIdx.x / LPK + y * (256 / LPK), left - 1), e = ke;
    kx[y] = bf16x8{};
    if (e < dk) {
      kx[y] = *reinterpret_cast<const bf16x8*>(p.proj + (t0 + tt) * d.ld + d.k0() + h * dk + e);
      if (TURNS) turn[y] = turn_of(p, e, pos0 + tt);
    }
  }
#pragma unroll
  for (int y = 0; y < NV; ++y) {
    const int tt = min((int)threadIdx.x / LPV + y * (256 / LPV), left - 1);
    vx[y] = bf16x8{};
    if (ve < dv) vx[y] = *reinterpret_cast<const bf16x8*>(p.proj + (t0 + tt) * d.ld + d.v0() + h * dv + ve);
  }
  if (w == 0) {
    float f = 0.f, i = -INFINITY, G, P;
    if (lane < left) log_gates(p, t0 + lane, h, f, i);
    run_sums(f, i, G, P);
    const float F = __shfl(G, 63, 64), b = F + __shfl(P, 63, 64);
    sw[lane] = expf(F - G + i - b);
    if (lane == 0) {
      float* sc = out + d.head();
      sc[0] = F;
      sc[1] = b;
      if (chunk == 0) sc[2] = d.gated && s.seen > 0 ? *head_max(p, s, h) : 0.f;
    }
  }
  __syncthreads();
#pragma unroll
  for (int y = 0; y < NK; ++y) {
    const int t = threadIdx.x / LPK + y * (256 / LPK), e = ke;
    if (e < kp) {
      float v[8];
      turned<TURNS>(kx[y], turn[y], v);
      const float f = sw[t];
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] = e < dk ? v[j] * f : 0.f;
      bf16x8 pl[3];
      split8<3>(v, pl);
#pragma unroll
      for (int k = 0; k < 3; ++k) *reinterpret_cast<bf16x8*>(lds + (k * kChunk + t) * ldk + e) = pl[k];
    }
  }
#pragma unroll
  for (int y = 0; y < NV; ++y) {
    const int t = threadIdx.x / LPV + y * (256 / LPV);
    if (ve < vp) *reinterpret_cast<bf16x8*>(sv + t * ldv + ve) = vx[y];
  }
  __syncthreads();
  bf16x8 a[KT][2][3];
#pragma unroll
  for (int r = 0; r < KT; ++r)
#pragma unroll
    for (int ks = 0; ks < 2; ++ks)
#pragma unroll
      for (int k = 0; k < 3; ++k)
        a[r][ks][k] = read_tokens(lds + (k * kChunk + 32 * ks) * ldk + min(16 * (w + 4 * r), kp - 16), ldk);
  for (int c = 0; c < vp; c += 16) {
    f32x4 acc[KT];
#pragma unroll
    for (int r = 0; r < KT; ++r) acc[r] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      const bf16x8 b = read_tokens(sv + 32 * ks * ldv + c, ldv);
#pragma unroll
      for (int k = 2; k >= 0; --k)
#pragma unroll
        for (int r = 0; r < KT; ++r) acc[r] = mfma_bf16(a[r][ks][k], b, acc[r]);
    }
    if (c + l15 < dv)
#pragma unroll
      for (int r = 0; r < KT; ++r) {
        const int row = 16 * (w + 4 * r) + 4 * g;  // (dk is a multiple of 8)
        if (row < dk)
#pragma unroll
          for (int j = 0; j < 4; ++j) (out + j * dv)[(uint32_t)(row * dv + c + l15)] = acc[r][j];
      }
  }
  if (d.gated)
    for (int e = threadIdx.x; e < dk; e += 256) {
      float n = 0.f;
      for (int t = 0; t < kChunk; ++t)
        n += ((float)lds[(2 * kChunk + t) * ldk + e] + (float)lds[(kChunk + t) * ldk + e]) + (float)lds[t * ldk + e];
      out[(int64_t)dk * dv + e] = n;
    }
}

// A thread: 4 neighbouring floats of a head's state (S, then n) over all chunks.
__global__ __launch_bounds__(256) void memory_chunk_walk_kernel(MemoryParams<bf16> p, ChunkWs ws) {
  const Seq s = seq_of(p, blockIdx.z);
  if (s.n <= 0) return;
  const MemoryDims& d = p.d;
  const int h = blockIdx.y, at = 4 * (blockIdx.x * 256 + threadIdx.x), hf = d.head();
  const int chunks = (s.n + kChunk - 1) / kChunk;
  const bool on = at < hf;
  const int64_t step = (int64_t)d.H * ws.floats;
  float* w0 = ws.at(s, blockIdx.z, 0, h, d.H);
  float* sc = w0 + hf;
  float* st = head_state(p, s, h) + at;
  f32x4 S = {0.f, 0.f, 0.f, 0.f};
  if (on && s.seen > 0) S = *reinterpret_cast<const f32x4*>(st);
  float m = sc[2];
  constexpr int U = 8;  // chunks in flight
  for (int c0 = 0; c0 < chunks; c0 += U) {
    f32x4 x[U];
    float F[U], b[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int64_t c = (int64_t)min(c0 + u, chunks - 1) * step;
      if (on) x[u] = *reinterpret_cast<const f32x4*>(w0 + c + at);
      F[u] = sc[c];
      b[u] = sc[c + 1];
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (c0 + u >= chunks) break;
      const int64_t c = (int64_t)(c0 + u) * step;
      if (on) *reinterpret_cast<f32x4*>(w0 + c + at) = S;
      if (blockIdx.x == 0 && threadIdx.x == 0 && c0 + u > 0) sc[c + 2] = m;
      const float now = fmaxf(F[u] + m, b[u]);
      S = expf(F[u] + m - now) * S + expf(b[u] - now) * x[u];
      m = now;
    }
  }
  if (on) *reinterpret_cast<f32x4*>(st) = S;
  if (d.gated && blockIdx.x == 0 && threadIdx.x == 0) *head_max(p, s, h) = m;
}

// which products of the pieces of two operands are kept: all of one number with an exact one, else the six largest
template <int NA, int NB, typename F>
__device__ __forceinline__ void piece_products(F&& f) {
#pragma unroll
  for (int order = 2; order >= 0; --order)  // the smallest first
#pragma unroll
    for (int a = 0; a < NA; ++a) {
      const int b = order - a;
      if (b >= 0 && b < NB) f(a, b);
    }
}

// Eight waves. KS: key dims / 32 (zero-filled), PL: pieces of a q or k element (1: bfloat16 as projected), LPU lanes per token
// in the norm. First the 64 x 64 matrix A, wave (block of 16 queries, half of the blocks of 16 keys), then every wave takes 16
// columns of the head.
template <int KS, int PL, int LPU>
__global__ __launch_bounds__(512, PL == 1 && LPU <= 16 ? 4 : 2) void memory_chunk_out_kernel(MemoryParams<bf16> p, ChunkWs ws) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  constexpr int ldq = 32 * KS + kPadRow, lda = kChunk + kPadRow;
  __shared__ float rows[2][kChunk], s_alpha[kChunk], s_inv[kChunk], s_row[kChunk], s_col[kChunk], s_floor[kChunk];
  const Seq s = seq_of(p, blockIdx.z);
  const int chunk = blockIdx.x, h = blockIdx.y, left = s.n - chunk * kChunk;
  if (left <= 0) return;
  const MemoryDims& d = p.d;
  const int dk = d.dk, dv = d.dv, vp = (dv + 15) / 16 * 16, ldv = vp + kPadRow, ldo = dv + 4;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, l15 = lane & 15, g = lane >> 4;
  const int64_t t0 = s.q0 + chunk * kChunk;
  const int pos0 = s.seen + chunk * kChunk;
  const float* front = ws.at(s, blockIdx.z, chunk, h, d.H);
  bf16* sq = reinterpret_cast<bf16*>(smem);      // [PL][64][ldq]
  bf16* sa = sq + PL * kChunk * ldq;             // [3][64][lda]
  bf16* sv = sa + 3 * kChunk * lda;              // [64][ldv]
  float* so = reinterpret_cast<float*>(smem);    // [64][ldo], when q and A have been read
  const float scale = 1.f / sqrtf((float)dk);
  constexpr bool TURNS = PL > 1;
  // Everything a thread reads is requested at once (the keys' cosines apart). Rows past the end repeat the last one: they are
  // not stored.
  constexpr int NQ = (KS + 1) / 2, NV = LPU / 8, NG = LPU / 8;
  const int ge = 8 * (threadIdx.x % LPU);  // columns of v and of the gate
  bf16x8 qx[NQ], vx[NV], kx[2][KS], gx[NG];
  Turn turn[NQ];
#pragma unroll
  for (int y = 0; y < NQ; ++y) {
    const int x = threadIdx.x + 512 * y, t = x / (4 * KS), e = 8 * (x - t * 4 * KS), tt = min(t, left - 1);
    qx[y] = bf16x8{};
    if (e < dk && t < kChunk) {
      qx[y] = *reinterpret_cast<const bf16x8*>(p.proj + (t0 + tt) * d.ld + h * dk + e);
      if (TURNS) turn[y] = turn_of(p, e, pos0 + tt);
    }
  }
  float f = 0.f, i = -INFINITY;
  if (w == 0 && lane < left) log_gates(p, t0 + lane, h, f, i);
  const int ib = w & 3, half = w >> 2;  // blocks of 16 queries; of 16 keys
#pragma unroll
  for (int y = 0; y < 2; ++y)
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int jb = half + 2 * y, e = 32 * ks + 8 * g;
      kx[y][ks] = bf16x8{};
      if (jb <= ib && e < dk)
        kx[y][ks] = *reinterpret_cast<const bf16x8*>(p.proj + (t0 + min(16 * jb + l15, left - 1)) * d.ld + d.k0() + h * dk + e);
    }
#pragma unroll
  for (int y = 0; y < NV; ++y) {
    const int t = threadIdx.x / LPU + y * (512 / LPU);
    vx[y] = bf16x8{};
    if (ge < dv) vx[y] = *reinterpret_cast<const bf16x8*>(p.proj + (t0 + min(t, left - 1)) * d.ld + d.v0() + h * dv + ge);
  }
  float S0[KS][8];
  // rows of the state in front, one of columns c .. c + 15 (rows past dk: any others, q is zero there)
  auto state_at = [&](int c, int ks, float (&x)[8]) {
    const uint32_t at = min(32 * ks + 8 * g, dk - 8) * dv + min(c + l15, dv - 1);
#pragma unroll
    for (int j = 0; j < 8; ++j) x[j] = (front + j * dv)[at];
  };
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) state_at(16 * w, ks, S0[ks]);
#pragma unroll
  for (int y = 0; y < NG; ++y) {
    const int t = threadIdx.x / LPU + y * (512 / LPU);
    gx[y] = bf16x8{};
    if (ge < dv) gx[y] = *reinterpret_cast<const bf16x8*>(p.proj + (t0 + min(t, left - 1)) * d.ld + d.g0() + h * dv + ge);
  }
#pragma unroll
  for (int y = 0; y < NQ; ++y) {
    const int x = threadIdx.x + 512 * y, t = x / (4 * KS), e = 8 * (x - t * 4 * KS);
    if (t < kChunk) {
      float v[8];
      turned<TURNS>(qx[y], turn[y], v);
      if (TURNS && e >= dk)
#pragma unroll
        for (int j = 0; j < 8; ++j) v[j] = 0.f;
      bf16x8 pl[PL];
      split8<PL>(v, pl);
#pragma unroll
      for (int k = 0; k < PL; ++k) *reinterpret_cast<bf16x8*>(sq + (k * kChunk + t) * ldq + e) = pl[k];
    }
  }
#pragma unroll
  for (int y = 0; y < NV; ++y) {
    const int t = threadIdx.x / LPU + y * (512 / LPU);
    if (ge < vp) *reinterpret_cast<bf16x8*>(sv + t * ldv + ge) = vx[y];
  }
  if (w == 0) {  // factors of token `lane`
    float G, P;
    run_sums(f, i, G, P);
    const float m_front = front[d.head() + 2], m = G + fmaxf(m_front, P);
    s_alpha[lane] = expf(G + m_front - m) * scale;
    s_row[lane] = G - m;
    s_col[lane] = i - G;
    s_floor[lane] = expf(-m);
  }
  __syncthreads();
  {
    bf16x8 qf[KS][PL];
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int k = 0; k < PL; ++k)
        qf[ks][k] = *reinterpret_cast<const bf16x8*>(sq + (k * kChunk + 16 * ib + l15) * ldq + 32 * ks + 8 * g);
    const float fi = s_row[16 * ib + l15];
    float sum = 0.f;
#pragma unroll
    for (int y = 0; y < 2; ++y) {
      const int jb = half + 2 * y;
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
      if (jb <= ib) {
        const int tt = min(16 * jb + l15, left - 1);
        Turn kt[KS];
        if constexpr (TURNS)
#pragma unroll
          for (int ks = 0; ks < KS; ++ks) kt[ks] = turn_of(p, 32 * ks + 8 * g, pos0 + tt);
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
          bf16x8 kf[PL];
          if constexpr (TURNS) {
            float v[8];
            turned<true>(kx[y][ks], kt[ks], v);
            split8<PL>(v, kf);
          } else {
            kf[0] = kx[y][ks];
          }
          piece_products<PL, PL>([&](int a, int b) { acc = mfma_bf16(kf[a], qf[ks][b], acc); });
        }
      }
      // lane: query 16 ib + l15, keys 16 jb + 4 g + r
      float a[4];
      const f32x4 fj = *reinterpret_cast<const f32x4*>(s_col + 16 * jb + 4 * g);
#pragma unroll
      for (int r = 0; r < 4; ++r) {  // (missing keys: a factor of zero)
        const int j = 16 * jb + 4 * g + r;
        a[r] = j <= 16 * ib + l15 ? acc[r] * scale * __expf(fi + fj[r]) : 0.f;
        sum += a[r];
      }
      float rest[4] = {a[0], a[1], a[2], a[3]};
#pragma unroll
      for (int k = 0; k < 3; ++k) {
        bf16x4 v;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          v[r] = (bf16)rest[r];
          rest[r] -= (float)v[r];
        }
        *reinterpret_cast<bf16x4*>(sa + (k * kChunk + 16 * ib + l15) * lda + 16 * jb + 4 * g) = v;
      }
    }
    sum += __shfl_xor(sum, 16, 64);
    sum += __shfl_xor(sum, 32, 64);
    if (g == 0) rows[half][16 * ib + l15] = sum;
  }
  __syncthreads();
  if (d.gated) {  // eight lanes a query
    const int t = threadIdx.x >> 3;
    const float* n = front + (int64_t)dk * dv;
    float nq = 0.f;
    for (int e = threadIdx.x & 7; e < dk; e += 8) {
      float q = 0.f;
#pragma unroll
      for (int k = PL - 1; k >= 0; --k) q += (float)sq[(k * kChunk + t) * ldq + e];
      nq += n[e] * q;
    }
    nq = group_sum<8>(nq) * s_alpha[t] + rows[0][t] + rows[1][t];
    if ((threadIdx.x & 7) == 0) s_inv[t] = 1.f / (fmaxf(fabsf(nq), s_floor[t]) + kFloorEps);
  } else if (threadIdx.x < kChunk) {
    s_inv[threadIdx.x] = 1.f;
  }
  constexpr int kMaxTiles = LPU > 16 ? 2 : 1;  // dv <= 8 LPU
  f32x4 O[kMaxTiles][4];
#pragma unroll
  for (int x = 0; x < kMaxTiles; ++x) {
    const int c = 16 * (w + 8 * x);
#pragma unroll
    for (int b = 0; b < 4; ++b) O[x][b] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (c >= dv) continue;
    if (x > 0)
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) state_at(c, ks, S0[ks]);
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      bf16x8 sf[3];
      split8<3>(S0[ks], sf);
#pragma unroll
      for (int b = 0; b < 4; ++b) {
        bf16x8 qf[PL];
#pragma unroll
        for (int k = 0; k < PL; ++k)
          qf[k] = *reinterpret_cast<const bf16x8*>(sq + (k * kChunk + 16 * b + l15) * ldq + 32 * ks + 8 * g);
        piece_products<3, PL>([&](int a, int k) { O[x][b] = mfma_bf16(sf[a], qf[k], O[x][b]); });
      }
    }
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      O[x][b] *= s_alpha[16 * b + l15];
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        if (2 * ks > b) continue;
        const bf16x8 vf = read_tokens(sv + 32 * ks * ldv + c, ldv);
#pragma unroll
        for (int k = 2; k >= 0; --k) {
          const bf16* ap = sa + (k * kChunk + 16 * b + l15) * lda + 32 * ks + 4 * g;
          const bf16x8 af = __builtin_shufflevector(*reinterpret_cast<const bf16x4*>(ap),
                                                    *reinterpret_cast<const bf16x4*>(ap + 16), 0, 1, 2, 3, 4, 5, 6, 7);
          O[x][b] = mfma_bf16(vf, af, O[x][b]);
        }
      }
    }
  }
  __syncthreads();
  // lane: query 16 b + l15, columns c + 4 g + r
#pragma unroll
  for (int x = 0; x < kMaxTiles; ++x) {
    const int c = 16 * (w + 8 * x) + 4 * g;
    if (c < dv)
#pragma unroll
      for (int b = 0; b < 4; ++b) *reinterpret_cast<f32x4*>(so + (16 * b + l15) * ldo + c) = O[x][b] * s_inv[16 * b + l15];
  }
  __syncthreads();
  float nw[8] = {1.f, 1.f, 1.f, 1.f, 1.f, 1.f, 1.f, 1.f};
  if (ge < dv && p.norm != nullptr) Vec8<float>::load(p.norm + h * dv + ge, nw);
#pragma unroll
  for (int y = 0; y < NG; ++y) {
    const int t = threadIdx.x / LPU + y * (512 / LPU);
    const bool on = t < left && ge < dv;
    float o[8], ss = 0.f;
    if (on) {
      Vec8<float>::load(so + t * ldo + ge, o);
#pragma unroll
      for (int x = 0; x < 8; ++x) ss += o[x] * o[x];
    }
    ss = group_sum<LPU>(ss);
    if (!on) continue;
    const float rs = 1.f / sqrtf(ss / (float)dv + p.eps);
#pragma unroll
    for (int x = 0; x < 8; ++x) o[x] *= rs * nw[x] * gate_act<bf16>((float)gx[y][x], p.act);
    Vec8<bf16>::store(p.out + (t0 + t) * p.ldo + h * dv + ge, o);
  }
}

// ---------------------------------------------------------------------------------------------------------------
bool dims_ok(const MemoryDims& d) {
  return d.H >= 1 && d.H <= 65535 && d.dk >= 1 && d.dk <= 512 && d.dv >= 1 && d.dv <= 65536 && d.rot >= 0 && d.rot % 2 == 0 &&
         d.rot <= d.dk && d.ld >= (int64_t)d.width();
}

bool chunk_ok(int dtype, int dk, int dv) {
  return dtype == kBF16 && dk % 8 == 0 && dv % 8 == 0 && dk <= 128 && dv <= 256;
}
int chunk_floats(int dk, int dv, int gated) { return MemoryDims{1, dk, dv, 0, gated, 0}.head() + 4; }

template <typename K>
int allow_lds(K* kernel, int bytes) {
  if (bytes > 158 * 1024) return hipErrorInvalidValue;
  return bytes > 48 * 1024 ? hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 158 * 1024)
                           : hipSuccess;
}

template <int KT, bool TURNS, int LPV>
int launch_chunk_sum_as(const MemoryParams<bf16>& p, const ChunkWs& ws, dim3 grid, hipStream_t st) {
  static const int attr = allow_lds(memory_chunk_sum_kernel<KT, TURNS, LPV>, 158 * 1024);
  if (attr) return attr;
  const int kp = (p.d.dk + 15) / 16 * 16, vp = (p.d.dv + 15) / 16 * 16;
  const size_t lds = sizeof(bf16) * kChunk * (3 * (kp + kPadRow) + vp + kPadRow);
  hipLaunchKernelGGL((memory_chunk_sum_kernel<KT, TURNS, LPV>), grid, dim3(256), lds, st, p, ws);
  return hipGetLastError();
}
template <int KT, bool TURNS>
int launch_chunk_sum(const MemoryParams<bf16>& p, const ChunkWs& ws, dim3 grid, hipStream_t st) {
  if (p.d.dv <= 64) return launch_chunk_sum_as<KT, TURNS, 8>(p, ws, grid, st);
  if (p.d.dv <= 128) return launch_chunk_sum_as<KT, TURNS, 16>(p, ws, grid, st);
  return launch_chunk_sum_as<KT, TURNS, 32>(p, ws, grid, st);
}

template <int KS, int PL, int LPU>
int launch_chunk_out(const MemoryParams<bf16>& p, const ChunkWs& ws, dim3 grid, hipStream_t st) {
  static const int attr = allow_lds(memory_chunk_out_kernel<KS, PL, LPU>, 158 * 1024);
  if (attr) return attr;
  const int vp = (p.d.dv + 15) / 16 * 16;
  const size_t ops = sizeof(bf16) * kChunk * (PL * (32 * KS + kPadRow) + 3 * (kChunk + kPadRow) + vp + kPadRow);
  const size_t res = sizeof(float) * kChunk * (p.d.dv + 4), lds = ops > res ? ops : res;
  hipLaunchKernelGGL((memory_chunk_out_kernel<KS, PL, LPU>), grid, dim3(512), lds, st, p, ws);
  return hipGetLastError();
}

template <int KS, int PL>
int launch_chunk_out_as(const MemoryParams<bf16>& p, const ChunkWs& ws, dim3 grid, hipStream_t st) {
  if (p.d.dv <= 64) return launch_chunk_out<KS, PL, 8>(p, ws, grid, st);
  if (p.d.dv <= 128) return launch_chunk_out<KS, PL, 16>(p, ws, grid, st);
  return launch_chunk_out<KS, PL, 32>(p, ws, grid, st);
}

int launch_chunks(const MemoryParams<bf16>& p, float* base, int n_seqs, int max_new, hipStream_t st) {
  const ChunkWs ws{base, chunk_floats(p.d.dk, p.d.dv, p.d.gated)};
  const dim3 grid((max_new + kChunk - 1) / kChunk, p.d.H, n_seqs);
  const bool turns = p.d.rot > 0;
  const int sum = p.d.dk <= 64 ? (turns ? launch_chunk_sum<1, true>(p, ws, grid, st) : launch_chunk_sum<1, false>(p, ws, grid, st))
                               : (turns ? launch_chunk_sum<2, true>(p, ws, grid, st) : launch_chunk_sum<2, false>(p, ws, grid, st));
  if (sum) return sum;
  hipLaunchKernelGGL(memory_chunk_walk_kernel, dim3((p.d.head() / 4 + 255) / 256, p.d.H, n_seqs), dim3(256), 0, st, p, ws);
  if (const hipError_t e = hipGetLastError()) return e;
  const int ks = p.d.dk <= 32 ? 1 : p.d.dk <= 64 ? 2 : 4;
  if (turns) {
    if (ks == 1) return launch_chunk_out_as<1, 3>(p, ws, grid, st);
    if (ks == 2) return launch_chunk_out_as<2, 3>(p, ws, grid, st);
    return launch_chunk_out_as<4, 3>(p, ws, grid, st);
  }
  if (ks == 1) return launch_chunk_out_as<1, 1>(p, ws, grid, st);
  if (ks == 2) return launch_chunk_out_as<2, 1>(p, ws, grid, st);
  return launch_chunk_out_as<4, 1>(p, ws, grid, st);
}

template <typename T>
int launch_serial(const MemoryParams<T>& p, int n_seqs, int max_new, hipStream_t st) {
  const int dk = p.d.dk;
  if (p.d.gated) {
    hipLaunchKernelGGL(memory_gates_kernel<T>, dim3(p.d.H, n_seqs), dim3(64), 0, st, p);
    if (const hipError_t e = hipGetLastError()) return e;
  }
  const dim3 grid((p.d.dv + 63) / 64, p.d.H, n_seqs);
#define HDS_MS(RR) hipLaunchKernelGGL((memory_scan_kernel<T, RR>), grid, dim3(256), 0, st, p)
  if (dk <= 32) HDS_MS(8); else if (dk <= 64) HDS_MS(16); else if (dk <= 128) HDS_MS(32); else if (dk <= 256) HDS_MS(64);
  else HDS_MS(128);
#undef HDS_MS
  if (const hipError_t e = hipGetLastError()) return e;
  hipLaunchKernelGGL(memory_out_kernel<T>, dim3(((int64_t)max_new * p.d.H + 3) / 4, n_seqs), dim3(256), 0, st, p);
  return hipGetLastError();
}

// threads and rows a thread of memory_step; 0: the kernel does not take these sizes
int step_shape(int dk, int dv, int& nt) {
  if (dv % 4 || dv > 1024) return 0;
  nt = (int64_t)dk * dv <= 4096 ? 256 : 1024;
  if (dv / 4 > nt) nt = 1024;
  const int rg = nt / (dv / 4), rows = (dk + rg - 1) / rg;
  return rows <= 16 ? rows : 0;
}
size_t step_lds(int dk, int dv, int nt) {
  const int cq = dv / 4, rg = nt / cq;
  const bool fold = (cq & (cq - 1)) == 0 && cq <= 64;
  return sizeof(float) * (2 * (size_t)dk + (size_t)(fold ? nt / 64 : rg) * dv);
}

template <typename T>
int launch_step(const MemoryParams<T>& p, int n_seqs, hipStream_t st) {
  int nt = 0;
  const int rows = step_shape(p.d.dk, p.d.dv, nt);
  const size_t lds = rows ? step_lds(p.d.dk, p.d.dv, nt) : 0;
  if (rows == 0 || lds > 60 * 1024 || p.slot_stride % 4 || (uintptr_t)p.state % 16) return hipErrorInvalidValue;
#define HDS_MT(RR, NN) hipLaunchKernelGGL((memory_step_kernel<T, RR, NN>), dim3(p.d.H, n_seqs), dim3(NN), lds, st, p)
#define HDS_MTN(NN)                                                                                      \
  {                                                                                                      \
    if (rows <= 1) HDS_MT(1, NN); else if (rows <= 2) HDS_MT(2, NN); else if (rows <= 4) HDS_MT(4, NN); \
    else if (rows <= 8) HDS_MT(8, NN); else HDS_MT(16, NN);                                              \
  }
  if (nt == 256) HDS_MTN(256) else HDS_MTN(1024)
#undef HDS_MTN
#undef HDS_MT
  return hipGetLastError();
}

template <typename T>
bool params_ok(const MemoryParams<T>& p, int n_seqs) {
  return dims_ok(p.d) && n_seqs <= 65535 && p.proj && p.state && p.slots && p.seq_meta && p.out &&
         p.ldo >= (int64_t)p.d.H * p.d.dv && p.slot_stride >= p.d.states() && (p.d.rot == 0 || (p.cos_t && p.sin_t)) &&
         (p.d.gated ? p.bi != nullptr && p.bf != nullptr && p.cap > 0.f : p.log_decay != nullptr);
}

}  // namespace

// heads of these sizes run memory_step (else single tokens run like portions)
HDS_EXPORT int hds_memory_step_ok(int dk, int dv) {
  int nt = 0;
  return dk >= 1 && dv >= 1 && step_shape(dk, dv, nt) > 0 && step_lds(dk, dv, nt) <= 60 * 1024;
}

// floats of the chunk scan's scratch memory per chunk and head (a step of n tokens has up to n / 64 + n_seqs chunks);
// 0: heads of these sizes and this type are scanned token by token
HDS_EXPORT int hds_memory_chunk_floats(int dtype, int dk, int dv, int gated) {
  return chunk_ok(dtype, dk, dv) ? chunk_floats(dk, dv, gated) : 0;
}
HDS_EXPORT int hds_memory_chunk_tokens() { return kChunk; }

// single != 0: the sequences' one new token each. Otherwise portions of at most max_new tokens, by chunks with the scratch
// memory `chunks` (the sequences ascend in the step's rows; proj and out rows 16-byte aligned), or with null token by token
// with o [tokens, H, dv] and, for the gated kind, coef [tokens, H, 4] as scratch memory. Gated kind: log_decay null, else bi, bf
// null. rot 0: no rotation. norm may be null. act: 0 sigmoid, 1 silu.
HDS_EXPORT int hds_memory(int dtype, int single, const void* proj, int64_t ld, const float* log_decay, const float* bi,
                          const float* bf, float cap, const float* cos_t, const float* sin_t, int rot, const float* norm,
                          int act, float* state, int64_t slot_stride, const int* slots, const int* seq_meta,
                          const int* seqs, float* coef, float* o, float* chunks, void* out, int64_t ldo, int n_seqs,
                          int max_new, int H, int dk, int dv, float eps, hipStream_t st) {
  if (n_seqs <= 0 || max_new <= 0) return 0;
  const int gated = log_decay == nullptr;
  const MemoryDims d{H, dk, dv, rot, gated, ld};
#define HDS_MP(TT)                                                                                                     \
  MemoryParams<TT> { d, (const TT*)proj, log_decay, bi, bf, cap, cos_t, sin_t, norm, act, state, slot_stride, slots, \
                     seq_meta, seqs, coef, o, (TT*)out, ldo, eps }
  const auto run = [&](const auto& p) -> int {
    if (!params_ok(p, n_seqs)) return hipErrorInvalidValue;
    if (single) return launch_step(p, n_seqs, st);
    if (o == nullptr || (gated && coef == nullptr)) return hipErrorInvalidValue;
    return launch_serial(p, n_seqs, max_new, st);
  };
  if (dtype == kBF16) {
    const auto p = HDS_MP(bf16);
    if (single || chunks == nullptr) return run(p);
    if (!params_ok(p, n_seqs) || !chunk_ok(dtype, dk, dv) || ld % 8 || ldo % 8 || (uintptr_t)proj % 16 ||
        (uintptr_t)out % 16 || slot_stride % 4 || (uintptr_t)state % 16)
      return hipErrorInvalidValue;
    return launch_chunks(p, chunks, n_seqs, max_new, st);
  }
  if (dtype == kF32) return run(HDS_MP(float));
#undef HDS_MP
  return hipErrorInvalidValue;
}
