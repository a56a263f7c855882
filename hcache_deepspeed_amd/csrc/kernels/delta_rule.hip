// Gated delta rule of a recurrent mixer over ragged batches. A head h carries a 32-bit state S [dk, dv]; per token
//
//   x      = silu(conv(x))                        for the channels of q, k and v: causal, depthwise, `taps` wide
//   q, k   = q / |q| * dk^(-1/2),  k / |k|        |x| = sqrt(sum(x^2) + 1e-6); query / key head h / (H / G)
//   beta   = sigmoid(b),  g = exp(-exp(A) * softplus(a + dt))
//   u      = beta (v - g S^T k),  S' = g S + k u^T,  o = S'^T q
//   out    = o / sqrt(mean(o^2) + eps) * w * silu(gate)
//
// One projection row holds, column block by column block, q [G dk] | k [G dk] | v [H dv] | gate [H dv], another (or the same
// one further on) b [H] | a [H].
// A sequence's slot holds S of all heads and then the convolution's last inputs as a ring: the input of position p is
// entry p % taps, [taps, C] with C = 2 G dk + H dv. (With taps - 1 of them in use, a step of one token reads other entries
// than it writes, so the workgroups of heads that share a key head need no order among them.) A sequence whose `seen` is
// 0 starts from zero whatever the slot holds.
//
// Single tokens run one kernel, a workgroup per (sequence, head): delta_step. Portions run delta_conv (convolutions,
// factors of the unit norms, log decays and betas), a scan over the tokens, and delta_out (norm and gate of the heads).
// The scan goes token by token (delta_scan: short portions, 32-bit engines, any sizes) or by chunks on the matrix cores
// (delta_chunk_prep, delta_chunk_state, delta_chunk_out).
#include <type_traits>

#include "hds_common.h"

namespace {
using namespace hds;

constexpr float kUnitEps = 1e-6f;

__device__ __forceinline__ float sigmoid_f(float x) {
  const float e = expf(-fabsf(x)), r = 1.f / (1.f + e);
  return x >= 0.f ? r : e * r;
}
__device__ __forceinline__ float silu_f(float x) { return x * sigmoid_f(x); }
__device__ __forceinline__ float softplus_f(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
// of activations and output gates (rounded to T)
template <typename T>
__device__ __forceinline__ float silu_act(float x) {
  if constexpr (sizeof(T) == 2) return x * __builtin_amdgcn_rcpf(1.f + __expf(-x));
  return silu_f(x);
}
template <typename T>
__device__ __forceinline__ float rounded(float x) { return to_f(from_f<T>(x)); }

struct DeltaDims {
  int H, G, dk, dv, taps;
  int64_t ld;  // row stride of the projection
  __device__ __host__ __forceinline__ int k0() const { return G * dk; }
  __device__ __host__ __forceinline__ int v0() const { return 2 * G * dk; }
  __device__ __host__ __forceinline__ int C() const { return 2 * G * dk + H * dv; }      // convolved channels
  __device__ __host__ __forceinline__ int width() const { return 2 * G * dk + 2 * H * dv; }
  __device__ __host__ __forceinline__ int64_t states() const { return (int64_t)H * dk * dv; }
};

template <typename T>
struct DeltaParams {
  DeltaDims d;
  const T* proj;        // [tokens, d.ld]
  const T* ba;          // [tokens, ldba]
  int64_t ldba;
  const float* cw;      // [taps, C], the last row is the current token's
  const float* a_log;   // [H]
  const float* dt;      // [H]
  const float* norm;    // [dv]
  float* state;         // [slots] x slot_stride
  int64_t slot_stride;
  const int* slots;
  const int* seq_meta;  // [sequences][3] = {first row, new tokens, seen}
  const int* seqs;      // the sequences this launch works on; null: 0, 1, ..
  T* y;                 // [tokens, C] convolved channels
  float* rn;            // [tokens, 2 G] factors of q (with dk^(-1/2)) and k
  float* gb;            // [tokens, H, 2] log decay, beta
  float* o;             // [tokens, H, dv] read-outs
  T* out;               // [tokens, ldo]
  int64_t ldo;
  int n_tok;
  float eps;
};

struct Seq {
  int q0, n, seen, slot;
};
template <typename T>
__device__ __forceinline__ Seq seq_of(const DeltaParams<T>& p, int i) {
  const int s = p.seqs != nullptr ? p.seqs[i] : i;
  return {p.seq_meta[3 * s], p.seq_meta[3 * s + 1], p.seq_meta[3 * s + 2], p.slots[s]};
}

// ---------------------------------------------------------------------------------------------------------------
// convolutions, unit norms, decays
// ---------------------------------------------------------------------------------------------------------------
// heads in channel order: G query heads, G key heads, H value heads
__device__ __forceinline__ void unit_of(const DeltaDims& d, int u, int& c0, int& width) {
  width = u < 2 * d.G ? d.dk : d.dv;
  c0 = u < 2 * d.G ? u * d.dk : d.v0() + (u - 2 * d.G) * d.dv;
}

template <typename T>
__device__ __forceinline__ void write_gates(const DeltaParams<T>& p, const Seq& s, int t0, int rows) {
  for (int i = threadIdx.x; i < rows * p.d.H; i += blockDim.x) {
    const int t = s.q0 + t0 + i / p.d.H, h = i % p.d.H;
    const T* row = p.ba + (int64_t)t * p.ldba;
    float* gb = p.gb + 2 * ((int64_t)t * p.d.H + h);
    gb[0] = -expf(p.a_log[h]) * softplus_f(to_f(row[p.d.H + h]) + p.dt[h]);
    gb[1] = sigmoid_f(to_f(row[h]));
  }
}

template <typename T>
__device__ __forceinline__ void write_factor(const DeltaParams<T>& p, int t, int u, float ss) {
  if (u < 2 * p.d.G)
    p.rn[(int64_t)t * 2 * p.d.G + u] = 1.f / sqrtf(ss + kUnitEps) * (u < p.d.G ? 1.f / sqrtf((float)p.d.dk) : 1.f);
}

// The workgroup of a sequence's first tokens is the only one that reads the ring (R >= taps - 1) and writes it last.
// LPU lanes a head, 8 channels each; M >= taps - 1 rows of history in registers (dk, dv, ld, C multiples of 8)
template <typename T, int LPU, int M>
__global__ __launch_bounds__(256) void delta_conv8_kernel(DeltaParams<T> p, int R) {
  const Seq s = seq_of(p, blockIdx.z);
  const int start = blockIdx.x * R;
  if (start >= s.n) return;
  const int rows = min(R, s.n - start), m = p.d.taps - 1;
  if (blockIdx.y == 0) write_gates(p, s, start, rows);
  const int u = blockIdx.y * (256 / LPU) + threadIdx.x / LPU;
  const bool live = u < 2 * p.d.G + p.d.H;
  int c0, width;
  unit_of(p.d, live ? u : 0, c0, width);
  const int e = 8 * (threadIdx.x % LPU);
  const bool ok = live && e < width;
  const int c = c0 + (ok ? e : 0);
  float* ring = p.state + (int64_t)s.slot * p.slot_stride + p.d.states() + c;
  const T* in = p.proj + (int64_t)s.q0 * p.d.ld + c;
  const int C = p.d.C();
  float w[M + 1][8], hist[M + 1][8];  // [k]: k + 1 back for hist, k back for w
#pragma unroll
  for (int k = 0; k <= M; ++k) {
#pragma unroll
    for (int i = 0; i < 8; ++i) w[k][i] = hist[k][i] = 0.f;
    if (k <= m) Vec8<float>::load(p.cw + (int64_t)(m - k) * C + c, w[k]);
    if (k < m) {
      const int i0 = start - 1 - k, pos = s.seen + i0;
      if (i0 >= 0) Vec8<T>::load(in + (int64_t)i0 * p.d.ld, hist[k]);
      else if (pos >= 0) Vec8<float>::load(ring + (int64_t)(pos % p.d.taps) * C, hist[k]);
    }
  }
  constexpr int U = 4;  // rows in flight, and as many requested ahead
  float nx[U][8];
  auto fetch = [&](int r) {
#pragma unroll
    for (int k = 0; k < U; ++k) Vec8<T>::load(in + (int64_t)(start + min(r + k, rows - 1)) * p.d.ld, nx[k]);
  };
  fetch(0);
  for (int r0 = 0; r0 < rows; r0 += U) {
    float xs[U][8];
#pragma unroll
    for (int k = 0; k < U; ++k)
#pragma unroll
      for (int i = 0; i < 8; ++i) xs[k][i] = nx[k][i];
    if (r0 + U < rows) fetch(r0 + U);
#pragma unroll
    for (int b = 0; b < U; ++b) {
      float y[8], ss = 0.f;
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        float a = w[0][i] * xs[b][i];
#pragma unroll
        for (int k = 0; k < M; ++k) a += w[k + 1][i] * hist[k][i];
        y[i] = rounded<T>(silu_act<T>(rounded<T>(a)));
        ss += ok ? y[i] * y[i] : 0.f;
      }
      const int t = s.q0 + start + r0 + b;
      ss = group_sum<LPU>(ss);
      if (ok && r0 + b < rows) {
        Vec8<T>::store(p.y + (int64_t)t * C + c, y);
        if (e == 0) write_factor(p, t, u, ss);
      }
#pragma unroll
      for (int k = M - 1; k > 0; --k)
#pragma unroll
        for (int i = 0; i < 8; ++i) hist[k][i] = hist[k - 1][i];
#pragma unroll
      for (int i = 0; i < 8; ++i) hist[0][i] = xs[b][i];
    }
  }
  if (blockIdx.x == 0 && ok)
    for (int i0 = max(s.n - m, 0); i0 < s.n; ++i0) {
      float v[8];
      Vec8<T>::load(in + (int64_t)i0 * p.d.ld, v);
      Vec8<float>::store(ring + (int64_t)((s.seen + i0) % p.d.taps) * C, v);
    }
}

// any sizes: one wave a head
template <typename T>
__global__ __launch_bounds__(256) void delta_conv_kernel(DeltaParams<T> p, int R) {
  const Seq s = seq_of(p, blockIdx.z);
  const int start = blockIdx.x * R;
  if (start >= s.n) return;
  const int rows = min(R, s.n - start), m = p.d.taps - 1;
  if (blockIdx.y == 0) write_gates(p, s, start, rows);
  const int u = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (u >= 2 * p.d.G + p.d.H) return;
  int c0, width;
  unit_of(p.d, u, c0, width);
  float* ring = p.state + (int64_t)s.slot * p.slot_stride + p.d.states();
  const T* in = p.proj + (int64_t)s.q0 * p.d.ld;
  const int C = p.d.C();
  for (int r = 0; r < rows; ++r) {
    float ss = 0.f;
    for (int c = c0 + lane; c < c0 + width; c += 64) {
      float a = 0.f;
      for (int k = 0; k <= m; ++k) {
        const int i0 = start + r - k, pos = s.seen + i0;
        if (pos < 0) break;
        const float v = i0 >= 0 ? to_f(in[(int64_t)i0 * p.d.ld + c]) : ring[(int64_t)(pos % p.d.taps) * C + c];
        a += p.cw[(int64_t)(m - k) * C + c] * v;
      }
      const float y = rounded<T>(silu_act<T>(rounded<T>(a)));
      p.y[(int64_t)(s.q0 + start + r) * C + c] = from_f<T>(y);
      ss += y * y;
    }
    ss = wave_sum(ss);
    if (lane == 0) write_factor(p, s.q0 + start + r, u, ss);
  }
  if (blockIdx.x == 0)
    for (int c = c0 + lane; c < c0 + width; c += 64)
      for (int i0 = max(s.n - m, 0); i0 < s.n; ++i0)
        ring[(int64_t)((s.seen + i0) % p.d.taps) * C + c] = to_f(in[(int64_t)i0 * p.d.ld + c]);
}

// ---------------------------------------------------------------------------------------------------------------
// scan, token by token: a workgroup per 64 columns of one head's state, R rows of it in each wave's registers
// ---------------------------------------------------------------------------------------------------------------
constexpr int kScanTok = 8;  // tokens staged at a time

template <typename T, int R>
__global__ __launch_bounds__(256) void delta_scan_kernel(DeltaParams<T> p) {
  __shared__ float sq[2][kScanTok][4 * R], sk[2][kScanTok][4 * R];
  __shared__ float part[2][4][2][64];
  __shared__ float sg[2][kScanTok][3];  // decay, beta, k . q
  const Seq s = seq_of(p, blockIdx.z);
  if (s.n <= 0) return;
  const int h = blockIdx.y, hk = h / (p.d.H / p.d.G);
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int col = blockIdx.x * 64 + lane, dk = p.d.dk, dv = p.d.dv, C = p.d.C();
  const bool ok = col < dv;
  const int cc = ok ? col : dv - 1;
  float* st = p.state + (int64_t)s.slot * p.slot_stride + (int64_t)h * dk * dv + cc;
  float S[R];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int row = w * R + r;
    S[r] = s.seen > 0 && row < dk ? st[(int64_t)row * dv] : 0.f;
  }
  // unit vectors of kScanTok tokens; wave w prepares tokens w, w + 4, ..
  auto stage = [&](int buf, int t0) {
    for (int i = w; i < kScanTok; i += 4) {
      if (t0 + i >= s.n) break;
      const int64_t t = s.q0 + t0 + i;
      const T* y = p.y + t * C;
      const float rq = p.rn[t * 2 * p.d.G + hk], rk = p.rn[t * 2 * p.d.G + p.d.G + hk];
      float kq = 0.f;
      for (int e = lane; e < 4 * R; e += 64) {
        const float q = e < dk ? to_f(y[hk * dk + e]) * rq : 0.f;
        const float k = e < dk ? to_f(y[p.d.k0() + hk * dk + e]) * rk : 0.f;
        sq[buf][i][e] = q;
        sk[buf][i][e] = k;
        kq += k * q;
      }
      kq = wave_sum(kq);
      if (lane == 0) {
        sg[buf][i][0] = expf(p.gb[2 * (t * p.d.H + h)]);
        sg[buf][i][1] = p.gb[2 * (t * p.d.H + h) + 1];
        sg[buf][i][2] = kq;
      }
    }
  };
  stage(0, 0);
  __syncthreads();
  for (int t0 = 0; t0 < s.n; t0 += kScanTok) {
    const int buf = (t0 / kScanTok) & 1, nt = min(kScanTok, s.n - t0);
    if (t0 + kScanTok < s.n) stage(buf ^ 1, t0 + kScanTok);
    float vn = to_f(p.y[(int64_t)(s.q0 + t0) * C + p.d.v0() + h * dv + cc]);
    for (int i = 0; i < nt; ++i) {
      const float v = vn;
      if (i + 1 < nt) vn = to_f(p.y[(int64_t)(s.q0 + t0 + i + 1) * C + p.d.v0() + h * dv + cc]);
      float ks = 0.f, qs = 0.f;
#pragma unroll
      for (int r = 0; r < R; ++r) {
        ks += S[r] * sk[buf][i][w * R + r];
        qs += S[r] * sq[buf][i][w * R + r];
      }
      const int pb = (t0 + i) & 1;
      part[pb][w][0][lane] = ks;
      part[pb][w][1][lane] = qs;
      __syncthreads();  // one a token: the other part buffer is written next
      ks = part[pb][0][0][lane] + part[pb][1][0][lane] + part[pb][2][0][lane] + part[pb][3][0][lane];
      qs = part[pb][0][1][lane] + part[pb][1][1][lane] + part[pb][2][1][lane] + part[pb][3][1][lane];
      const float g = sg[buf][i][0], u = sg[buf][i][1] * (v - g * ks);
#pragma unroll
      for (int r = 0; r < R; ++r) S[r] = g * S[r] + sk[buf][i][w * R + r] * u;
      if (w == 0 && ok) p.o[((int64_t)(s.q0 + t0 + i) * p.d.H + h) * dv + col] = g * qs + sg[buf][i][2] * u;
    }
    __syncthreads();
  }
  if (ok)
#pragma unroll
    for (int r = 0; r < R; ++r)
      if (w * R + r < dk) st[(int64_t)(w * R + r) * dv] = S[r];
}

// ---------------------------------------------------------------------------------------------------------------
// scan by chunks of 64 tokens
// ---------------------------------------------------------------------------------------------------------------
// With G_i the sum of the log decays of a chunk's tokens up to i, S the state before the chunk and u_i as above,
//
//   (1 + L) U = beta V - diag(beta e^G) K S,      L_ij = beta_i e^(G_i - G_j) k_i . k_j   (j < i)
//   O         = diag(e^G) Q S + A U,              A_ij = e^(G_i - G_j) q_i . k_j          (j <= i)
//   S        <- e^G_last S + sum_j e^(G_last - G_j) k_j u_j^T
//
// delta_chunk_prep, all chunks at once: 16 x 16 blocks of -L below the diagonal, the inverses of the diagonal blocks of
// 1 + L, the blocks of A, and the factors per token. delta_chunk_state, a wave per 16 columns of a head's state: walks the
// chunks with S in registers and leaves every chunk's S and U. delta_chunk_out, all chunks at once: O, its norm and its
// gate. Everything is 32-bit: q and k are bfloat16 up to a 32-bit factor per token, so products among them are exact on
// the bfloat16 matrix cores; S and U enter their products with q and k as sums of three bfloat16 numbers (24 bits); the
// blocks of L and A multiply U on the 32-bit matrix cores.
//
// An accumulator tile (lane: column l & 15, rows 4 (l >> 4) + r) is the right operand of the next product as it is, if the
// left operand takes its contraction index in the same order: f32 step r contracts rows 4 (l >> 4) + r of a 16-row block,
// a bf16 step over tokens the rows 4 (l >> 4) .. + 3 of two blocks. The rows of S are dealt to the tiles such that a bf16
// step over them takes 8 neighbours.
constexpr int kChunk = 64, kBlocks = 10;                // lower 16 x 16 blocks
constexpr int kWalkFloats = kBlocks * 256 + 5 * kChunk; // what the walk reads: blocks of L, factors
constexpr int kFixedFloats = kWalkFloats + kBlocks * 256;
__device__ __forceinline__ constexpr int block_at(int b, int j) { return b * (b + 1) / 2 + j; }

// Scratch memory of a chunk and head: blocks of L | factors [5][64] | blocks of A, then per 16 columns of the state its
// 2 KS tiles and U's 4 tiles as the lanes hold them. The chunks of sequence i start at q0 / 64 + i (they do not overlap).
struct ChunkWs {
  float* base;
  int64_t floats;  // per chunk and head
  __device__ __forceinline__ float* at(const Seq& s, int i, int chunk, int h, int H) const {
    return base + ((int64_t)(s.q0 / kChunk + i + chunk) * H + h) * floats;
  }
};
__device__ __host__ __forceinline__ constexpr int strip_floats(int ks) { return (2 * ks + 4) * 256; }

// KS: key dims / 32 (dk a multiple of 8, zero-filled to 32 KS)
template <int KS>
__global__ __launch_bounds__(256) void delta_chunk_prep_kernel(DeltaParams<bf16> p, ChunkWs ws) {
  __shared__ float sl[4][16][17];
  const Seq s = seq_of(p, blockIdx.z);
  const int chunk = blockIdx.x, h = blockIdx.y;
  if (chunk * kChunk >= s.n) return;
  const DeltaDims& d = p.d;
  const int hk = h / (d.H / d.G), C = d.C();
  const int lane = threadIdx.x & 63, b = threadIdx.x >> 6, l15 = lane & 15, g = lane >> 4;
  const int left = s.n - chunk * kChunk;  // tokens from the chunk's start on
  const int64_t t0 = s.q0 + chunk * kChunk;
  float* out = ws.at(s, blockIdx.z, chunk, h, d.H);
  float G = 0.f, beta = 0.f, rq = 0.f, rk = 0.f;  // of token `lane`; missing tokens change nothing
  if (lane < left) {
    const float* gb = p.gb + 2 * ((t0 + lane) * d.H + h);
    G = gb[0];
    beta = gb[1];
    rq = p.rn[(t0 + lane) * 2 * d.G + hk];
    rk = p.rn[(t0 + lane) * 2 * d.G + d.G + hk];
  }
#pragma unroll
  for (int o = 1; o < 64; o <<= 1) {
    const float v = __shfl_up(G, o, 64);
    if (lane >= o) G += v;
  }
  const float last = __shfl(G, 63, 64);
  if (b == 0) {
    float* sc = out + kBlocks * 256 + lane;
    const float eg = expf(G);
    sc[0] = beta * eg * rk;
    sc[kChunk] = beta;
    sc[2 * kChunk] = eg * rq;
    sc[3 * kChunk] = expf(last - G) * rk;
    sc[4 * kChunk] = expf(last);
  }
  auto frag = [&](int blk, int base, int ks) {  // rows 16 blk + l15 of q or k
    const int e = 32 * ks + 8 * g;
    bf16x8 v = {};
    if (e < d.dk) v = *reinterpret_cast<const bf16x8*>(p.y + (t0 + min(16 * blk + l15, left - 1)) * C + base + hk * d.dk + e);
    return v;
  };
  bf16x8 kb[KS], qb[KS];
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) {
    kb[ks] = frag(b, d.k0(), ks);
    qb[ks] = frag(b, 0, ks);
  }
  float Gi[4], bi[4], qi[4], ki[4];  // of the rows 16 b + 4 g + r
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int i = 16 * b + 4 * g + r;
    Gi[r] = __shfl(G, i, 64);
    bi[r] = __shfl(beta, i, 64);
    qi[r] = __shfl(rq, i, 64);
    ki[r] = __shfl(rk, i, 64);
  }
  for (int j = 0; j <= b; ++j) {
    f32x4 kk = {0.f, 0.f, 0.f, 0.f}, qk = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const bf16x8 kj = frag(j, d.k0(), ks);
      kk = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kb[ks], kj, kk, 0, 0, 0);
      qk = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qb[ks], kj, qk, 0, 0, 0);
    }
    const float Gj = __shfl(G, 16 * j + l15, 64), kj = __shfl(rk, 16 * j + l15, 64);
    float* m1 = out + block_at(b, j) * 256 + l15;
    float* am = m1 + kWalkFloats;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = 4 * g + r;
      const bool below = j < b || row > l15, on = below || row == l15;
      const float e = on ? expf(Gi[r] - Gj) * kj : 0.f;
      am[row * 16] = e * qi[r] * qk[r];
      const float l = below ? bi[r] * e * ki[r] * kk[r] : 0.f;
      if (j < b) m1[row * 16] = -l;
      else sl[b][row][l15] = l;
    }
  }
  __syncthreads();
  if (lane < 16) {  // column l15 of (1 + L_bb)^-1 by forward substitution
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float v = i == l15 ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < i; ++j) v -= sl[b][i][j] * x[j];
      x[i] = v;
      out[block_at(b, b) * 256 + i * 16 + l15] = v;
    }
  }
}

// row of S in register r of accumulator tile t: 8 neighbouring rows of two tiles are the 8 contraction indices a lane of the
// bfloat16 products holds
__device__ __forceinline__ int state_row(int t, int g, int r) { return 32 * (t >> 1) + 8 * g + 4 * (t & 1) + r; }

// Transposed LDS reads as inline asm: in front of the builtin the compiler waits for every direct load and store under way
// (it cannot tell that they go elsewhere). tr_wait is due before the values are used.
template <int OFF>
__device__ __forceinline__ bf16x4 read_tr4(const char* a) {
  bf16x4 r;
  asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(r) : "v"((uint32_t)(uintptr_t)a), "n"(OFF) : "memory");
  return r;
}
__device__ __forceinline__ void tr_wait(bf16x4& a, bf16x4& b) {
  asm volatile("s_waitcnt lgkmcnt(0)" : "+v"(a), "+v"(b) : : "memory");
}
__device__ __forceinline__ f32x4 mfma_bf16(const bf16x8& a, const bf16x8& b, const f32x4& c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

// Eight numbers as sums of three bfloat16 numbers (24 bits), in 12 steps of a few instructions, to lie between matrix
// products
struct Split {
  u32x4 bits[3];  // high, middle, low
  float r[8];
  template <int STEP>
  __device__ __forceinline__ void step(const f32x4& a, const f32x4& b) {
    typedef __bf16 bf16x2 __attribute__((ext_vector_type(2)));
    typedef float f32x2 __attribute__((ext_vector_type(2)));
    constexpr int i = STEP / 3, k = STEP % 3;
    const f32x2 x = k > 0 ? f32x2{r[2 * i], r[2 * i + 1]}
                          : (i < 2 ? f32x2{a[2 * i & 3], a[(2 * i & 3) + 1]} : f32x2{b[2 * i & 3], b[(2 * i & 3) + 1]});
    const uint32_t v = __builtin_bit_cast(uint32_t, __builtin_convertvector(x, bf16x2));
    bits[k][i] = v;
    if (k < 2) {
      r[2 * i] = x[0] - __builtin_bit_cast(float, v << 16);
      r[2 * i + 1] = x[1] - __builtin_bit_cast(float, v & 0xFFFF0000u);
    }
  }
  __device__ __forceinline__ bf16x8 p(int k) const { return __builtin_bit_cast(bf16x8, bits[k]); }
  __device__ __forceinline__ void all(const f32x4& a, const f32x4& b);
};
__device__ __forceinline__ void split_step(Split& s, int i, const f32x4& a, const f32x4& b) {
  switch (i) {  // i: a constant after unrolling
    case 0: s.step<0>(a, b); break;
    case 1: s.step<1>(a, b); break;
    case 2: s.step<2>(a, b); break;
    case 3: s.step<3>(a, b); break;
    case 4: s.step<4>(a, b); break;
    case 5: s.step<5>(a, b); break;
    case 6: s.step<6>(a, b); break;
    case 7: s.step<7>(a, b); break;
    case 8: s.step<8>(a, b); break;
    case 9: s.step<9>(a, b); break;
    case 10: s.step<10>(a, b); break;
    case 11: s.step<11>(a, b); break;
    default: break;
  }
}

__device__ __forceinline__ void Split::all(const f32x4& a, const f32x4& b) {
#pragma unroll
  for (int i = 0; i < 12; ++i) split_step(*this, i, a, b);
}

// LDS image of a chunk, filled by direct loads (a wave instruction writes 64 lanes x 16 bytes in a row, so rows have no
// padding; 16-byte pieces are swapped within a row instead, by the row number): k as 64 rows of 256 bytes, 64 / Z columns
// of v as 64 rows, the chunk's blocks and factors as they are.
constexpr int kTileV = 16384;
static_assert((4 * kWalkFloats + 4095) / 4096 * 4096 <= 4 * kFixedFloats, "reads past the entry");
template <int Z>
struct ChunkTile {
  static constexpr int kPieces = 8 / Z, kRowsV = 64 / kPieces;  // of v: pieces of a row, rows of a wave instruction
  static constexpr int kW = kTileV + 64 * 16 * kPieces, kBytes = kW + (4 * kWalkFloats + 4095) / 4096 * 4096;
  __device__ __forceinline__ static int swap(int row) { return Z == 1 ? row & 7 : (row >> 2) & 3; }
  __device__ __forceinline__ static int off(int row, int piece) { return (row * kPieces + (piece ^ swap(row))) * 16; }
};
__device__ __forceinline__ int piece_of(int row) { return ((row & 3) << 2) | ((row >> 2) & 3); }
__device__ __forceinline__ int row_off(int row, int piece) { return row * 256 + 16 * (piece ^ piece_of(row)); }
__device__ __forceinline__ void direct_load(const void* src, char* dst) {
  __builtin_amdgcn_global_load_lds((__attribute__((address_space(1))) const void*)src,
                                   (__attribute__((address_space(3))) void*)dst, 16, 0, 0);
}

// Z waves share 16 columns, each with its part of the key dims: they add up their parts of K S through LDS and then work out
// the same U. (A wave's vector instructions do not run under its own matrix products, and there are fewer strips of columns
// than SIMDs.) FULL: dk == 32 KS and dv a multiple of 64 (no lane of a direct load is left out, which would split the
// schedule).
template <int KS, bool FULL>
__global__ __launch_bounds__(256, 1) void delta_chunk_state_kernel(DeltaParams<bf16> p, ChunkWs ws) {
  extern __shared__ __attribute__((aligned(1024))) char lds[];  // three chunks: this one, the next, the one on its way
  const Seq s = seq_of(p, blockIdx.z);
  if (s.n <= 0) return;
  const DeltaDims& d = p.d;
  const int h = blockIdx.y, hk = h / (d.H / d.G), C = d.C(), dv = d.dv;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, l15 = lane & 15, g = lane >> 4;
  constexpr int Z = KS > 1 ? 2 : 1, KZ = KS / Z, kStrips = 4 / Z;
  using Tile = ChunkTile<Z>;
  const int strip = w % kStrips, z = w / kStrips;
  const int c0 = blockIdx.x * 16 * kStrips, col = c0 + 16 * strip + l15;
  const bool active = FULL || c0 + 16 * strip < dv, ok = FULL || col < dv;
  float* st = p.state + (int64_t)s.slot * p.slot_stride + (int64_t)h * d.dk * dv;
  f32x4 S[2 * KZ];
#pragma unroll
  for (int t = 0; t < 2 * KZ; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = state_row(2 * KZ * z + t, g, r);
      S[t][r] = s.seen > 0 && ok && row < d.dk ? st[(int64_t)row * dv + col] : 0.f;
    }
  // Rows past the end repeat the last one: their factors are zero. Key columns past dk stay zero: a row of S there would
  // take part otherwise.
  const bf16* yk = p.y + (int64_t)s.q0 * C + d.k0() + hk * d.dk;
  const bf16* yv = p.y + (int64_t)s.q0 * C + d.v0() + h * dv + c0;
  constexpr int kLoadsV = 2 / Z, kLoadsW = (4 * kWalkFloats + 4095) / 4096;
  constexpr int kLoads = 4 + kLoadsV + kLoadsW;  // direct loads a wave issues for a chunk
  static_assert(kLoadsW == 3, "the last three go out late");
  auto fetch_one = [&](int buffer, int chunk, int i) {
    char* tile = lds + buffer * Tile::kBytes;
    const int last = s.n - 1 - chunk * kChunk;
    const int64_t at = (int64_t)chunk * kChunk * C;
    if (i < 4) {  // 4 rows of k an instruction
      const int n = 4 * w + i, row = 4 * n + (lane >> 4), e = 8 * ((lane & 15) ^ piece_of(row));
      if (FULL || e < d.dk) direct_load(yk + at + (uint32_t)(min(row, last) * C + e), tile + n * 1024);
    } else if (i < 4 + kLoadsV) {
      const int n = kLoadsV * w + i - 4, row = n * Tile::kRowsV + lane / Tile::kPieces;
      const int e = 8 * (lane % Tile::kPieces ^ Tile::swap(row));
      if (FULL || c0 + e < dv) direct_load(yv + at + (uint32_t)(min(row, last) * C + e), tile + kTileV + n * 1024);
    } else {
      const char* cw = reinterpret_cast<const char*>(ws.at(s, blockIdx.z, chunk, h, d.H)) + 16 * lane;
      const int n = 4 * (i - 4 - kLoadsV) + w;  // (the last one reads into the blocks of A)
      direct_load(cw + n * 1024, tile + Tile::kW + n * 1024);
    }
  };
  auto fetch = [&](int buffer, int chunk) {
#pragma unroll
    for (int i = 0; i < kLoads; ++i) fetch_one(buffer, chunk, i);
  };
  const int chunks = (s.n + kChunk - 1) / kChunk;
  if (!FULL && d.dk < 32 * KS) {
    for (int i = threadIdx.x; i < 3 * Tile::kBytes / 16; i += 256) reinterpret_cast<u32x4*>(lds)[i] = u32x4{};
    __syncthreads();
  }
  // Offsets of this lane's reads in a tile. Row blocks and halves are 16-row steps, which leave the swap of the pieces as
  // it is; another k step or key block flips bits of the offset.
  const int q = l15 >> 2, pp = l15 & 3;
  const int row_at = row_off(l15, g) ^ (64 * KZ * z);         // ^ 64 ks; + 4096 b
  const int col_at = row_off(4 * g + q, pp) ^ (64 * KZ * z);  // ^ 64 (t >> 1); + 8 (t & 1), + 4096 per 16 tokens
  const int v_at = kTileV + Tile::off(4 * g + q, 2 * strip + (pp >> 1)) + 8 * (pp & 1);  // + kBlockV b
  constexpr int kBlockV = 16 * 16 * Tile::kPieces;
  char* parts = lds + 3 * Tile::kBytes + 16 * lane;           // [wave][4 tiles]
  fetch(0, 0);
  fetch(1, min(1, chunks - 1));
  Split sp[2];
  sp[0].all(S[0], S[1]);
  __syncthreads();
  int buffer = 0;
  for (int ch = 0; ch < chunks; ++ch) {
    const char* tile = lds + buffer * Tile::kBytes;
    const int free = buffer == 0 ? 2 : buffer - 1;      // was read in the step before
    const int next = min(ch + 2, chunks - 1);           // (the last one again: no branch)
    if (active) {
      const char* cw = tile + Tile::kW;
      auto block = [&](int b, int j) {
        return *reinterpret_cast<const f32x4*>(cw + block_at(b, j) * 1024 + l15 * 64 + 16 * g);
      };
      auto factor = [&](int k, int b) {
        return *reinterpret_cast<const f32x4*>(cw + kBlocks * 1024 + k * 4 * kChunk + 64 * b + 16 * g);
      };
      // Operands are read from LDS one step ahead of the products that use them, products of different accumulators follow
      // one another, and the splits of the next operands lie between them: the scheduling barriers keep it so.
      bf16x4 v[4];
      v[0] = read_tr4<0>(tile + v_at);
      v[1] = read_tr4<kBlockV>(tile + v_at);
      v[2] = read_tr4<2 * kBlockV>(tile + v_at);
      v[3] = read_tr4<3 * kBlockV>(tile + v_at);
      tr_wait(v[0], v[1]);
      tr_wait(v[2], v[3]);
      bf16x8 kf[2][4];
      auto rows = [&](int ks, bf16x8 (&kk)[4]) {
#pragma unroll
        for (int b = 0; b < 4; ++b) kk[b] = *reinterpret_cast<const bf16x8*>(tile + (row_at ^ (64 * ks)) + 4096 * b);
      };
      rows(0, kf[0]);
      float* keep_s = ws.at(s, blockIdx.z, ch, h, d.H) + kFixedFloats + (int64_t)(c0 / 16 + strip) * strip_floats(KS) + 4 * lane;
      f32x4 U[4];  // K S, then u
#pragma unroll
      for (int b = 0; b < 4; ++b) U[b] = f32x4{0.f, 0.f, 0.f, 0.f};
      f32x4 M1[4][4], f0[4], f1[4], f3[4];  // [row block][column block]
      const float keep = *reinterpret_cast<const float*>(cw + kBlocks * 1024 + 16 * kChunk);
#pragma unroll
      for (int ks = 0; ks < KZ; ++ks) {
        __builtin_amdgcn_sched_barrier(0);
        if (ks + 1 < KZ) {
          rows(ks + 1, kf[(ks + 1) & 1]);
        } else {
#pragma unroll
          for (int b = 0; b < 4; ++b) {
            f0[b] = factor(0, b);
            f1[b] = factor(1, b);
            f3[b] = factor(3, b);
          }
#pragma unroll
          for (int b = 0; b < 4; ++b)
#pragma unroll
            for (int j = 0; j <= b; ++j) M1[b][j] = block(b, j);
        }
#pragma unroll
        for (int i = 0; i < 12; ++i) {  // the smallest piece first
          __builtin_amdgcn_sched_barrier(0);
          U[i & 3] = mfma_bf16(kf[ks & 1][i & 3], sp[ks & 1].p(2 - i / 4), U[i & 3]);
          if (ks + 1 < KZ) split_step(sp[(ks + 1) & 1], i, S[2 * ks + 2], S[2 * ks + 3]);
          // loads and stores are spread over the step: the wave would wait for a queue that is full
          constexpr int kEvery = 12 * KZ / (kLoads - 3);
          const int n = 12 * ks + i;
          if (n % kEvery == kEvery - 1 && n / kEvery < kLoads - 3) fetch_one(free, next, n / kEvery);
        }
      }
      __builtin_amdgcn_sched_barrier(0);
      if constexpr (Z == 2) {
#pragma unroll
        for (int b = 0; b < 4; ++b) *reinterpret_cast<f32x4*>(parts + (4 * w + b) * 1024) = U[b];
        asm volatile("s_waitcnt lgkmcnt(0)" : : : "memory");
        __builtin_amdgcn_s_barrier();
        asm volatile("" : : : "memory");
#pragma unroll
        for (int b = 0; b < 4; ++b) U[b] += *reinterpret_cast<const f32x4*>(parts + (4 * (w ^ 2) + b) * 1024);
      }
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int b = 0; b < 4; ++b)
#pragma unroll
        for (int r = 0; r < 4; ++r) U[b][r] = f1[b][r] * (float)v[b][r] - f0[b][r] * U[b][r];
      bf16x4 kt[2][2 * KZ][2];  // transposed k: all key dims of 32 tokens
      auto cols = [&](int hf) {
#pragma unroll
        for (int t = 0; t < 2 * KZ; ++t) {
          const char* p0 = tile + (col_at ^ (64 * (t >> 1)));
          kt[hf][t][0] = hf == 0 ? (t & 1 ? read_tr4<8>(p0) : read_tr4<0>(p0))
                                 : (t & 1 ? read_tr4<8200>(p0) : read_tr4<8192>(p0));
          kt[hf][t][1] = hf == 0 ? (t & 1 ? read_tr4<4104>(p0) : read_tr4<4096>(p0))
                                 : (t & 1 ? read_tr4<12296>(p0) : read_tr4<12288>(p0));
        }
      };
      auto key = [&](int hf, int t) {
        return __builtin_shufflevector(kt[hf][t][0], kt[hf][t][1], 0, 1, 2, 3, 4, 5, 6, 7);
      };
      Split up[2];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        __builtin_amdgcn_sched_barrier(0);
        if (j == 1) cols(0);
        __builtin_amdgcn_sched_barrier(0);
        f32x4 x = {0.f, 0.f, 0.f, 0.f}, y = x;
        x = __builtin_amdgcn_mfma_f32_16x16x4f32(M1[j][j][0], U[j][0], x, 0, 0, 0);
        y = __builtin_amdgcn_mfma_f32_16x16x4f32(M1[j][j][1], U[j][1], y, 0, 0, 0);
        x = __builtin_amdgcn_mfma_f32_16x16x4f32(M1[j][j][2], U[j][2], x, 0, 0, 0);
        y = __builtin_amdgcn_mfma_f32_16x16x4f32(M1[j][j][3], U[j][3], y, 0, 0, 0);
        U[j] = x + y;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
#pragma unroll
          for (int b = j + 1; b < 4; ++b) U[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(M1[b][j][r], U[j][r], U[b], 0, 0, 0);
          const int t = j == 0 ? r : (j == 1 ? 4 + r : 2 * KZ);  // S goes out, then decays
          if (t < 2 * KZ) {
            *reinterpret_cast<f32x4*>(keep_s + 256 * (2 * KZ * z + t)) = S[t];
            S[t] *= keep;
            __builtin_amdgcn_sched_barrier(0);
          }
        }
        if (Z == 1 || j / 2 == z) *reinterpret_cast<f32x4*>(keep_s + 256 * (2 * KS + j)) = U[j];
        U[j] *= f3[j];
        if (j == 2) up[0].all(U[0], U[1]);
      }
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int t = 0; t < 2 * KZ; ++t) tr_wait(kt[0][t][0], kt[0][t][1]);
      cols(1);
#pragma unroll
      for (int i = 0; i < 6 * KZ; ++i) {
        __builtin_amdgcn_sched_barrier(0);
        S[i % (2 * KZ)] = mfma_bf16(key(0, i % (2 * KZ)), up[0].p(2 - i / (2 * KZ)), S[i % (2 * KZ)]);
        if (KZ >= 2) split_step(up[1], i, U[2], U[3]);
        if (i % (2 * KZ) == 0) fetch_one(free, next, kLoads - 3 + i / (2 * KZ));
      }
      if (KZ < 2) up[1].all(U[2], U[3]);
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int t = 0; t < 2 * KZ; ++t) tr_wait(kt[1][t][0], kt[1][t][1]);
      // tiles 0 and 1 first: their sum is the first operand of the next chunk
#pragma unroll
      for (int i = 0; i < 6; ++i) S[i & 1] = mfma_bf16(key(1, i & 1), up[1].p(2 - i / 2), S[i & 1]);
      constexpr int R = 2 * KZ - 2;  // the other tiles
#pragma unroll
      for (int i = 0; i < 3 * R; ++i) {
        __builtin_amdgcn_sched_barrier(0);
        S[2 + i % (R > 0 ? R : 1)] = mfma_bf16(key(1, 2 + i % (R > 0 ? R : 1)), up[1].p(2 - i / (R > 0 ? R : 1)),
                                               S[2 + i % (R > 0 ? R : 1)]);
        if (i >= 2) split_step(sp[0], i - 2, S[0], S[1]);
      }
#pragma unroll
      for (int i = R > 0 ? 3 * R - 2 : 0; i < 12; ++i) split_step(sp[0], i, S[0], S[1]);
      __builtin_amdgcn_sched_barrier(0);
      // the next chunk's loads went out a step ago: all but this step's loads and stores have to be done
      asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)" : : "n"(kLoads + 2 * KZ + 4 / Z) : "memory");
    } else {
      fetch(free, next);
      if constexpr (Z == 2) __builtin_amdgcn_s_barrier();
      asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)" : : "n"(kLoads) : "memory");
    }
    __builtin_amdgcn_s_barrier();
    asm volatile("" : : : "memory");
    buffer = buffer == 2 ? 0 : buffer + 1;
  }
  if (ok)
#pragma unroll
    for (int t = 0; t < 2 * KZ; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = state_row(2 * KZ * z + t, g, r);
        if (row < d.dk) st[(int64_t)row * dv + col] = S[t][r];
      }
}

// O = diag(e^G) Q S + A U of a chunk and head, its norm and gate. Eight waves share the head's columns, 16 at a time; then
// LPU lanes a token, 8 columns each.
template <int KS, int LPU>
__global__ __launch_bounds__(512, 4) void delta_chunk_out_kernel(DeltaParams<bf16> p, ChunkWs ws) {
  extern __shared__ __attribute__((aligned(16))) float so[];  // [64][dv + 4]
  const Seq s = seq_of(p, blockIdx.z);
  const int chunk = blockIdx.x, h = blockIdx.y;
  const int left = s.n - chunk * kChunk;
  if (left <= 0) return;
  const DeltaDims& d = p.d;
  const int hk = h / (d.H / d.G), C = d.C(), dv = d.dv, ld = dv + 4;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, l15 = lane & 15, g = lane >> 4;
  const int64_t t0 = s.q0 + chunk * kChunk;
  const float* cw = ws.at(s, blockIdx.z, chunk, h, d.H);
  const int strips = (dv + 15) / 16;
  if (w < strips) {
    // rows past the end repeat the last one: they are not stored
    const bf16* qr[4];
#pragma unroll
    for (int b = 0; b < 4; ++b) qr[b] = p.y + (t0 + min(16 * b + l15, left - 1)) * C + hk * d.dk + 8 * g;
    for (int strip = w; strip < strips; strip += 8) {
      const float* sw = cw + kFixedFloats + (int64_t)strip * strip_floats(KS) + 4 * lane;
      f32x4 U[4], O[4], S[2][2];
      bf16x8 qf[2][4];
      auto fetch = [&](int ks) {
        S[ks & 1][0] = *reinterpret_cast<const f32x4*>(sw + 512 * ks);
        S[ks & 1][1] = *reinterpret_cast<const f32x4*>(sw + 512 * ks + 256);
#pragma unroll
        for (int b = 0; b < 4; ++b) {
          qf[ks & 1][b] = bf16x8{};
          if (32 * ks + 8 * g < d.dk) qf[ks & 1][b] = *reinterpret_cast<const bf16x8*>(qr[b] + 32 * ks);
        }
      };
      fetch(0);
#pragma unroll
      for (int b = 0; b < 4; ++b) O[b] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        if (ks + 1 < KS) {
          fetch(ks + 1);
        } else {
#pragma unroll
          for (int b = 0; b < 4; ++b) U[b] = *reinterpret_cast<const f32x4*>(sw + 256 * (2 * KS + b));
        }
        __builtin_amdgcn_sched_barrier(0);
        Split sp;
        sp.all(S[ks & 1][0], S[ks & 1][1]);
#pragma unroll
        for (int k = 2; k >= 0; --k)
#pragma unroll
          for (int b = 0; b < 4; ++b) O[b] = mfma_bf16(qf[ks & 1][b], sp.p(k), O[b]);
        __builtin_amdgcn_sched_barrier(0);
      }
      auto block = [&](int b, int j) {
        return *reinterpret_cast<const f32x4*>(cw + kWalkFloats + block_at(b, j) * 256 + l15 * 16 + 4 * g);
      };
      f32x4 A[2][4];
#pragma unroll
      for (int b = 0; b < 4; ++b) {
        A[0][b] = block(b, 0);
        O[b] *= *reinterpret_cast<const f32x4*>(cw + kBlocks * 256 + 2 * kChunk + 16 * b + 4 * g);
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) {
#pragma unroll
        for (int b = j + 1; b < 4; ++b) A[(j + 1) & 1][b] = block(b, j + 1);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
          for (int b = j; b < 4; ++b) O[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(A[j & 1][b][r], U[j][r], O[b], 0, 0, 0);
        __builtin_amdgcn_sched_barrier(0);
      }
      if (16 * strip + l15 < dv)
#pragma unroll
        for (int b = 0; b < 4; ++b)
#pragma unroll
          for (int r = 0; r < 4; ++r) so[(16 * b + 4 * g + r) * ld + 16 * strip + l15] = O[b][r];
    }
  }
  __syncthreads();
  const int e = 8 * (threadIdx.x % LPU);
  float nw[8];
  if (e < dv) Vec8<float>::load(p.norm + e, nw);
  for (int i = threadIdx.x / LPU; i < kChunk; i += 512 / LPU) {
    const bool on = i < left && e < dv;
    float o[8], gt[8], ss = 0.f;
    if (on) {
      Vec8<float>::load(so + i * ld + e, o);
      Vec8<bf16>::load(p.proj + (t0 + i) * d.ld + C + h * dv + e, gt);
#pragma unroll
      for (int x = 0; x < 8; ++x) ss += o[x] * o[x];
    }
    ss = group_sum<LPU>(ss);
    if (!on) continue;
    const float rs = 1.f / sqrtf(ss / (float)dv + p.eps);
#pragma unroll
    for (int x = 0; x < 8; ++x) o[x] *= rs * nw[x] * silu_act<bf16>(gt[x]);
    Vec8<bf16>::store(p.out + (t0 + i) * p.ldo + h * dv + e, o);
  }
}

// ---------------------------------------------------------------------------------------------------------------
// norm and gate of the heads
// ---------------------------------------------------------------------------------------------------------------
template <typename T>
__device__ __forceinline__ bool out_item(const DeltaParams<T>& p, int64_t item, int R, int& t, int& h) {
  const Seq s = seq_of(p, blockIdx.z);
  const int start = blockIdx.x * R;
  const int i = start + (int)(item / p.d.H);
  h = (int)(item % p.d.H);
  t = s.q0 + i;
  return i < min(s.n, start + R);
}

// LPU lanes a head, 8 values each; a workgroup takes R tokens
template <typename T, int LPU>
__global__ __launch_bounds__(256) void delta_out8_kernel(DeltaParams<T> p, int R) {
  const int e = 8 * (threadIdx.x % LPU), dv = p.d.dv;
  if (blockIdx.x * R >= seq_of(p, blockIdx.z).n) return;
  float nw[8];
  if (e < dv) Vec8<float>::load(p.norm + e, nw);
  for (int64_t item = threadIdx.x / LPU; item < (int64_t)R * p.d.H; item += 256 / LPU) {
    int t, h;
    const bool ok = out_item(p, item, R, t, h) && e < dv;
    float o[8], g[8], ss = 0.f;
    if (ok) {
      Vec8<float>::load(p.o + ((int64_t)t * p.d.H + h) * dv + e, o);
      Vec8<T>::load(p.proj + (int64_t)t * p.d.ld + p.d.C() + h * dv + e, g);
#pragma unroll
      for (int i = 0; i < 8; ++i) ss += o[i] * o[i];
    }
    ss = group_sum<LPU>(ss);
    if (!ok) continue;
    const float rs = 1.f / sqrtf(ss / (float)dv + p.eps);
#pragma unroll
    for (int i = 0; i < 8; ++i) o[i] *= rs * nw[i] * silu_act<T>(g[i]);
    Vec8<T>::store(p.out + (int64_t)t * p.ldo + h * dv + e, o);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void delta_out_kernel(DeltaParams<T> p, int R) {
  const int lane = threadIdx.x & 63, dv = p.d.dv;
  for (int64_t item = threadIdx.x >> 6; item < (int64_t)R * p.d.H; item += 4) {
    int t, h;
    if (!out_item(p, item, R, t, h)) break;
    const float* o = p.o + ((int64_t)t * p.d.H + h) * dv;
    const T* g = p.proj + (int64_t)t * p.d.ld + p.d.C() + h * dv;
    float ss = 0.f;
    for (int e = lane; e < dv; e += 64) ss += o[e] * o[e];
    const float rs = 1.f / sqrtf(wave_sum(ss) / (float)dv + p.eps);
    for (int e = lane; e < dv; e += 64)
      p.out[(int64_t)t * p.ldo + h * dv + e] = from_f<T>(o[e] * rs * p.norm[e] * silu_act<T>(to_f(g[e])));
  }
}

// ---------------------------------------------------------------------------------------------------------------
// one token per sequence: everything from the projection to the gated output in a workgroup per (head, sequence)
// ---------------------------------------------------------------------------------------------------------------
// A thread keeps 4 columns of RPT rows of S. S^T k and S^T q come from one pass over the old state:
// o = g S^T q + (k . q) u.
// Loads go out in the order their values are needed: the convolution's, then S, then the norm's and the gate's.
template <typename T, int RPT, int NT>
__global__ __launch_bounds__(NT, NT < 1024 ? 1 : (RPT <= 4 ? 8 : 4)) void delta_step_kernel(DeltaParams<T> p) {
  constexpr int NW = NT / 64;
  extern __shared__ float sm[];
  const DeltaDims& d = p.d;
  const int dk = d.dk, dv = d.dv, C = d.C(), cq = dv / 4;
  const int RG = NT / cq;                     // row groups
  const bool fold = (cq & (cq - 1)) == 0 && cq <= 64;  // the row groups of a wave reduce by lane exchange
  const int P = fold ? NW : RG;
  float* part = sm;                           // [P][2][dv]
  float* su = part + 2 * P * dv;              // [dv]
  float* so = su + dv;                        // [dv]
  float* sq = so + dv;                        // [dk], then k [dk] and v [dv]
  float* sk = sq + dk;
  float* sv = sk + dk;
  const int h = blockIdx.x, hk = h / (d.H / d.G);
  const Seq s = seq_of(p, blockIdx.y);
  if (s.n != 1) return;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int c4 = threadIdx.x % cq, rg = threadIdx.x / cq;
  const bool act = rg < RG;
  float* st = p.state + (int64_t)s.slot * p.slot_stride;
  float* Sp = st + ((int64_t)h * dk) * dv + 4 * c4;
  const T* row = p.proj + (int64_t)s.q0 * d.ld;
  float* ring = st + d.states();
  const int now = s.seen % d.taps;  // ring entry of this token
  constexpr int MT = 4;             // taps whose operands are requested together
  auto channel = [&](int i) {
    return i < dk ? hk * dk + i : (i < 2 * dk ? d.k0() + hk * dk + i - dk : d.v0() + h * dv + i - 2 * dk);
  };
  const int n_ch = 2 * dk + dv;
  const int c_first = channel(min((int)threadIdx.x, n_ch - 1));
  const bool few = d.taps <= MT;
  float cw[MT], hist[MT];
  if (few) {
#pragma unroll
    for (int k = 0; k < MT; ++k) {
      cw[k] = k < d.taps ? p.cw[(int64_t)(d.taps - 1 - k) * C + c_first] : 0.f;
      hist[k] = 0.f;
      if (k == 0) hist[k] = to_f(row[c_first]);
      else if (k < d.taps && s.seen >= k) hist[k] = ring[(int64_t)(now >= k ? now - k : now - k + d.taps) * C + c_first];
    }
  }
  const T* ba = p.ba + (int64_t)s.q0 * p.ldba + h;
  const float xb = to_f(ba[0]), xa = to_f(ba[d.H]), al = p.a_log[h], dt = p.dt[h];
  f32x4 S[RPT];
#pragma unroll
  for (int r = 0; r < RPT; ++r) {
    S[r] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int e = rg + r * RG;
    if (act && s.seen > 0 && e < dk) S[r] = *reinterpret_cast<const f32x4*>(Sp + (int64_t)e * dv);
  }
  const int o_first = min((int)threadIdx.x, dv - 1);
  const float nw = p.norm[o_first], og = to_f(row[C + h * dv + o_first]);
  const float beta = sigmoid_f(xb), g = expf(-expf(al) * softplus_f(xa + dt));
  // convolutions of this head's channels
  for (int i = threadIdx.x; i < n_ch; i += NT) {
    const int c = channel(i);
    float x, a;
    if (few && i == (int)threadIdx.x) {
      x = hist[0];
      a = cw[0] * x;
#pragma unroll
      for (int k = 1; k < MT; ++k) a += cw[k] * hist[k];
    } else {
      x = to_f(row[c]);
      a = p.cw[(int64_t)(d.taps - 1) * C + c] * x;
      for (int k = 1; k < d.taps; ++k)
        if (s.seen >= k)
          a += p.cw[(int64_t)(d.taps - 1 - k) * C + c] * ring[(int64_t)((s.seen - k) % d.taps) * C + c];
    }
    sq[i] = rounded<T>(silu_act<T>(rounded<T>(a)));
    if (i >= 2 * dk || h % (d.H / d.G) == 0) ring[(int64_t)now * C + c] = x;
  }
  __syncthreads();
  float qq = 0.f, kk = 0.f, kq = 0.f;
  for (int e = lane; e < dk; e += 64) {
    qq += sq[e] * sq[e];
    kk += sk[e] * sk[e];
    kq += sk[e] * sq[e];
  }
  const float rq = 1.f / sqrtf(wave_sum(qq) + kUnitEps) / sqrtf((float)dk), rk = 1.f / sqrtf(wave_sum(kk) + kUnitEps);
  kq = wave_sum(kq) * rq * rk;
  f32x4 ks = {0.f, 0.f, 0.f, 0.f}, qs = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int r = 0; r < RPT; ++r) {
    const int e = rg + r * RG;
    if (act && e < dk) {
      ks += S[r] * sk[e];
      qs += S[r] * sq[e];
    }
  }
  if (fold) {
    for (int off = cq; off < 64; off <<= 1)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        ks[i] += __shfl_xor(ks[i], off, 64);
        qs[i] += __shfl_xor(qs[i], off, 64);
      }
    if (lane < cq) {
      *reinterpret_cast<f32x4*>(part + (2 * w) * dv + 4 * c4) = ks;
      *reinterpret_cast<f32x4*>(part + (2 * w + 1) * dv + 4 * c4) = qs;
    }
  } else if (act) {
    *reinterpret_cast<f32x4*>(part + (2 * rg) * dv + 4 * c4) = ks;
    *reinterpret_cast<f32x4*>(part + (2 * rg + 1) * dv + 4 * c4) = qs;
  }
  __syncthreads();
  for (int c = threadIdx.x; c < dv; c += NT) {
    float a = 0.f, b = 0.f;
#pragma unroll 8
    for (int i = 0; i < P; ++i) {
      a += part[(2 * i) * dv + c];
      b += part[(2 * i + 1) * dv + c];
    }
    const float u = beta * (sv[c] - g * rk * a);
    su[c] = u;
    so[c] = g * rq * b + kq * u;
  }
  __syncthreads();
  if (act) {
    const f32x4 u = *reinterpret_cast<const f32x4*>(su + 4 * c4);
#pragma unroll
    for (int r = 0; r < RPT; ++r) {
      const int e = rg + r * RG;
      if (e < dk) *reinterpret_cast<f32x4*>(Sp + (int64_t)e * dv) = g * S[r] + (rk * sk[e]) * u;
    }
  }
  if (w * 64 < dv) {
    float ss = 0.f;
    for (int c = lane; c < dv; c += 64) ss += so[c] * so[c];
    const float rs = 1.f / sqrtf(wave_sum(ss) / (float)dv + p.eps);
    for (int c = threadIdx.x; c < dv; c += NT)
      p.out[(int64_t)s.q0 * p.ldo + h * dv + c] = from_f<T>(
          c == (int)threadIdx.x ? so[c] * rs * nw * silu_act<T>(og)
                                : so[c] * rs * p.norm[c] * silu_act<T>(to_f(row[C + h * dv + c])));
  }
}

// ---------------------------------------------------------------------------------------------------------------
template <typename T>
int launch_conv(const DeltaParams<T>& p, int n_seqs, int max_new, hipStream_t st) {
  const DeltaDims& d = p.d;
  int R = 16;
  if (R < d.taps - 1) R = d.taps - 1;
  const int units = 2 * d.G + d.H, w = d.dk > d.dv ? d.dk : d.dv;
  const int blocks = (max_new + R - 1) / R;
  if (d.dk % 8 || d.dv % 8 || d.ld % 8 || d.taps > 8 || w > 512 || p.slot_stride % 4 || (uintptr_t)p.state % 16 ||
      (uintptr_t)p.proj % 16 || d.states() % 4) {
    hipLaunchKernelGGL(delta_conv_kernel<T>, dim3(blocks, (units + 3) / 4, n_seqs), dim3(256), 0, st, p, R);
    return hipGetLastError();
  }
#define HDS_DC(L, MM)                                                                                              \
  hipLaunchKernelGGL((delta_conv8_kernel<T, L, MM>), dim3(blocks, (units + 256 / L - 1) / (256 / L), n_seqs),     \
                     dim3(256), 0, st, p, R)
#define HDS_DCM(L) { if (d.taps <= 4) HDS_DC(L, 3); else HDS_DC(L, 7); }
  if (w <= 64) HDS_DCM(8) else if (w <= 128) HDS_DCM(16) else if (w <= 256) HDS_DCM(32) else HDS_DCM(64)
#undef HDS_DCM
#undef HDS_DC
  return hipGetLastError();
}

template <typename T>
int launch_out(const DeltaParams<T>& p, int n_seqs, int max_new, hipStream_t st) {
  const int dv = p.d.dv, R = 4;
  const dim3 grid((max_new + R - 1) / R, 1, n_seqs);
  if (dv % 8 || dv > 512 || p.d.ld % 8 || p.d.C() % 8 || p.ldo % 8 || (uintptr_t)p.out % 16 || (uintptr_t)p.proj % 16) {
    hipLaunchKernelGGL(delta_out_kernel<T>, grid, dim3(256), 0, st, p, R);
    return hipGetLastError();
  }
#define HDS_DO(L) hipLaunchKernelGGL((delta_out8_kernel<T, L>), grid, dim3(256), 0, st, p, R)
  if (dv <= 64) HDS_DO(8); else if (dv <= 128) HDS_DO(16); else if (dv <= 256) HDS_DO(32); else HDS_DO(64);
#undef HDS_DO
  return hipGetLastError();
}

template <typename T>
int launch_scan(const DeltaParams<T>& p, int n_seqs, hipStream_t st) {
  const dim3 grid((p.d.dv + 63) / 64, p.d.H, n_seqs);
#define HDS_DS(RR) hipLaunchKernelGGL((delta_scan_kernel<T, RR>), grid, dim3(256), 0, st, p)
  const int dk = p.d.dk;
  if (dk <= 32) HDS_DS(8); else if (dk <= 64) HDS_DS(16); else if (dk <= 128) HDS_DS(32); else if (dk <= 256) HDS_DS(64);
  else HDS_DS(128);
#undef HDS_DS
  return hipGetLastError();
}

bool chunk_ok(int dtype, int dk, int dv) {
  return dtype == kBF16 && dk % 8 == 0 && dv % 8 == 0 && dk <= 128 && dv <= 512;
}
int chunk_ks(int dk) { return dk <= 32 ? 1 : dk <= 64 ? 2 : 4; }
int chunk_floats(int dk, int dv) { return kFixedFloats + (dv + 15) / 16 * strip_floats(chunk_ks(dk)); }

template <int KS, int LPU>
int launch_chunk_out(const DeltaParams<bf16>& p, const ChunkWs& ws, dim3 grid, hipStream_t st) {
  static const hipError_t attr = hipFuncSetAttribute((const void*)delta_chunk_out_kernel<KS, LPU>,
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
  if (attr != hipSuccess) return attr;
  hipLaunchKernelGGL((delta_chunk_out_kernel<KS, LPU>), grid, dim3(512), kChunk * (p.d.dv + 4) * sizeof(float), st, p, ws);
  return hipGetLastError();
}

template <int KS, bool FULL>
int launch_chunk_state(const DeltaParams<bf16>& p, const ChunkWs& ws, int n_seqs, hipStream_t st) {
  constexpr int Z = KS > 1 ? 2 : 1, lds = 3 * ChunkTile<Z>::kBytes + (Z > 1 ? 16384 : 0), cols = 64 / Z;
  static_assert(lds <= 160 * 1024, "LDS");
  static const hipError_t attr = hipFuncSetAttribute((const void*)delta_chunk_state_kernel<KS, FULL>,
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, lds);
  if (attr != hipSuccess) return attr;
  hipLaunchKernelGGL((delta_chunk_state_kernel<KS, FULL>), dim3((p.d.dv + cols - 1) / cols, p.d.H, n_seqs), dim3(256), lds, st, p,
                     ws);
  return hipGetLastError();
}

template <int KS>
int launch_chunks_as(const DeltaParams<bf16>& p, const ChunkWs& ws, int n_seqs, int max_new, hipStream_t st) {
  const dim3 grid((max_new + kChunk - 1) / kChunk, p.d.H, n_seqs);
  hipLaunchKernelGGL(delta_chunk_prep_kernel<KS>, grid, dim3(256), 0, st, p, ws);
  if (const hipError_t e = hipGetLastError()) return e;
  const bool full = p.d.dk == 32 * KS && p.d.dv % 64 == 0;
  if (const int e = full ? launch_chunk_state<KS, true>(p, ws, n_seqs, st) : launch_chunk_state<KS, false>(p, ws, n_seqs, st))
    return e;
  if (p.d.dv <= 64) return launch_chunk_out<KS, 8>(p, ws, grid, st);
  if (p.d.dv <= 128) return launch_chunk_out<KS, 16>(p, ws, grid, st);
  if (p.d.dv <= 256) return launch_chunk_out<KS, 32>(p, ws, grid, st);
  return launch_chunk_out<KS, 64>(p, ws, grid, st);
}

// the scan and what follows it
int launch_chunks(const DeltaParams<bf16>& p, float* base, int n_seqs, int max_new, hipStream_t st) {
  const ChunkWs ws{base, chunk_floats(p.d.dk, p.d.dv)};
  switch (chunk_ks(p.d.dk)) {
    case 1: return launch_chunks_as<1>(p, ws, n_seqs, max_new, st);
    case 2: return launch_chunks_as<2>(p, ws, n_seqs, max_new, st);
    default: return launch_chunks_as<4>(p, ws, n_seqs, max_new, st);
  }
}

// threads and rows a thread of delta_step; 0: the kernel does not take these sizes
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
  return sizeof(float) * (2 * (size_t)dk + 3 * dv + 2 * (size_t)(fold ? nt / 64 : rg) * dv);
}

template <typename T>
int launch_step(const DeltaParams<T>& p, int n_seqs, hipStream_t st) {
  int nt = 0;
  const int rows = step_shape(p.d.dk, p.d.dv, nt);
  const size_t lds = rows ? step_lds(p.d.dk, p.d.dv, nt) : 0;
  if (rows == 0 || lds > 64 * 1024 || p.slot_stride % 4 || (uintptr_t)p.state % 16) return hipErrorInvalidValue;
#define HDS_DT(RR, NN) hipLaunchKernelGGL((delta_step_kernel<T, RR, NN>), dim3(p.d.H, n_seqs), dim3(NN), lds, st, p)
#define HDS_DTN(NN)                                                                                      \
  {                                                                                                      \
    if (rows <= 1) HDS_DT(1, NN); else if (rows <= 2) HDS_DT(2, NN); else if (rows <= 4) HDS_DT(4, NN); \
    else if (rows <= 8) HDS_DT(8, NN); else HDS_DT(16, NN);                                              \
  }
  if (nt == 256) HDS_DTN(256) else HDS_DTN(1024)
#undef HDS_DTN
#undef HDS_DT
  return hipGetLastError();
}

bool dims_ok(const DeltaDims& d) {
  return d.H >= 1 && d.G >= 1 && d.H % d.G == 0 && d.dk >= 1 && d.dk <= 512 && d.dv >= 1 && d.taps >= 1 &&
         d.taps <= 256 && d.H <= 65535 && d.ld >= (int64_t)d.width();
}

}  // namespace

// heads of these sizes run delta_step (else single tokens run like portions)
HDS_EXPORT int hds_delta_step_ok(int dk, int dv) {
  int nt = 0;
  return dk >= 1 && dv >= 1 && step_shape(dk, dv, nt) > 0 && step_lds(dk, dv, nt) <= 64 * 1024;
}

// the sequences' one new token each
HDS_EXPORT int hds_delta_step(int dtype, const void* proj, int64_t ld, const void* ba, int64_t ldba, const float* cw, const float* a_log,
                              const float* dt, const float* norm, float* state, int64_t slot_stride, const int* slots,
                              const int* seq_meta, const int* seqs, void* out, int64_t ldo, int n_seqs, int H, int G,
                              int dk, int dv, int taps, float eps, hipStream_t st) {
  if (n_seqs <= 0) return 0;
  const DeltaDims d{H, G, dk, dv, taps, ld};
  if (!dims_ok(d) || !ba || ldba < 2 * H || n_seqs > 65535 || !state || !slots || ldo < (int64_t)H * dv ||
      slot_stride < d.states() + (int64_t)taps * d.C())
    return hipErrorInvalidValue;
#define HDS_DX(TT)                                                                                                 \
  return launch_step(DeltaParams<TT>{d, (const TT*)proj, (const TT*)ba, ldba, cw, a_log, dt, norm, state, slot_stride, slots, seq_meta, \
                                     seqs, nullptr, nullptr, nullptr, nullptr, (TT*)out, ldo, 0, eps}, n_seqs, st)
  if (dtype == kBF16) HDS_DX(bf16);
  if (dtype == kF32) HDS_DX(float);
#undef HDS_DX
  return hipErrorInvalidValue;
}

// floats of the chunk scan's scratch memory per chunk and head (a step of n tokens has up to n / 64 + n_seqs chunks);
// 0: heads of these sizes and this type are scanned token by token
HDS_EXPORT int hds_delta_chunk_floats(int dtype, int dk, int dv) {
  return chunk_ok(dtype, dk, dv) ? chunk_floats(dk, dv) : 0;
}
HDS_EXPORT int hds_delta_chunk_tokens() { return kChunk; }

// Portions of at most max_new tokens. y [tokens, C], rn [tokens, 2 G] and gb [tokens, H, 2] are scratch memory with a row
// for every token of the step. chunks: scratch memory of the scan by chunks (the sequences ascend in the step's rows; proj
// and out rows 16-byte aligned); null: token by token, with o [tokens, H, dv] as scratch memory.
HDS_EXPORT int hds_delta_scan(int dtype, const void* proj, int64_t ld, const void* ba, int64_t ldba, const float* cw, const float* a_log,
                              const float* dt, const float* norm, float* state, int64_t slot_stride, const int* slots,
                              const int* seq_meta, const int* seqs, void* y, float* rn, float* gb, float* o, float* chunks,
                              void* out, int64_t ldo, int n_seqs, int max_new, int H, int G, int dk, int dv, int taps, float eps,
                              hipStream_t st) {
  if (n_seqs <= 0 || max_new <= 0) return 0;
  const DeltaDims d{H, G, dk, dv, taps, ld};
  if (!dims_ok(d) || !ba || ldba < 2 * H || n_seqs > 65535 || !state || !slots || !y || !rn || !gb || ldo < (int64_t)H * dv ||
      slot_stride < d.states() + (int64_t)taps * d.C())
    return hipErrorInvalidValue;
#define HDS_DX(TT)                                                                                                   \
  {                                                                                                                  \
    const DeltaParams<TT> p{d, (const TT*)proj, (const TT*)ba, ldba, cw, a_log, dt, norm, state, slot_stride, slots, seq_meta, seqs,     \
                            (TT*)y, rn, gb, o, (TT*)out, ldo, 0, eps};                                               \
    if (int e = launch_conv(p, n_seqs, max_new, st)) return e;                                                       \
    return scan(p);                                                                                                  \
  }
  const auto scan = [&](const auto& p) -> int {
    if constexpr (std::is_same<decltype(p.proj), const bf16*>::value)
      if (chunks != nullptr) return launch_chunks(p, chunks, n_seqs, max_new, st);
    if (int e = launch_scan(p, n_seqs, st)) return e;
    return launch_out(p, n_seqs, max_new, st);
  };
  if (chunks == nullptr && o == nullptr) return hipErrorInvalidValue;
  if (chunks != nullptr && (!chunk_ok(dtype, dk, dv) || ld % 8 || ldo % 8 || (uintptr_t)proj % 16 || (uintptr_t)out % 16))
    return hipErrorInvalidValue;
  if (dtype == kBF16) HDS_DX(bf16)
  if (dtype == kF32) HDS_DX(float)
#undef HDS_DX
  return hipErrorInvalidValue;
}
