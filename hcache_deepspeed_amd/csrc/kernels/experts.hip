// Routed expert layers of the serving engine: router, choice of the experts, and the expert products of small steps.
//
//   z = W_router h                       (32-bit accumulation and result)
//   s = softmax(z) over the experts and the identity experts behind them, or sigmoid(z)
//   c = s + correction                   (decides, does not weigh)
//   groups of neighbours are ranked by their largest c, only the best `keep` of them take part
//   the `top` largest c are chosen; weight = s * scale, of an expert's output, or of its input: then the product's rows are
//   multiplied with it in front of the activation
//
// Steps of few tokens run the experts straight from the choices (experts_skinny_kernel: every chosen expert's weights
// are streamed once, whatever the number of tokens that chose it, the gated activation included). Longer steps sort
// the choices by expert (expert_sort_kernel, which also writes the tile list of the products) and run the grouped
// GEMM of grouped_gemm.hip, or its 32-bit counterpart here. Nothing of it needs the host.
#include "hds_common.h"

namespace {
using namespace hds;

// ---------------------------------------------------------------------------------------------------------------
// router
// ---------------------------------------------------------------------------------------------------------------
// logits[T, R] = x[T, K] . w[R, K]^T in 32-bit. A workgroup: 16 RT router rows x 16 tokens, its NW waves take every
// NW-th 32 of K (K % 32 == 0). mfma_f32_16x16x32_bf16 with A = router rows, B = tokens (accumulator column = token).
// Long steps use a large RT (the tokens are read once for most routers), short ones spread over workgroups.
template <int RT, int NW>
__global__ __launch_bounds__(64 * NW) void router_logits_kernel(const bf16* __restrict__ x, int64_t ldx,
                                                            const bf16* __restrict__ w, float* __restrict__ z,
                                                            int64_t ldz, int T, int R, int K) {
  __shared__ f32x4 red[NW - 1][RT][64];
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int r0 = blockIdx.x * 16 * RT, t0 = blockIdx.y * 16;
  const int kb = 8 * (lane >> 4);
  const bf16* wp[RT];
#pragma unroll
  for (int i = 0; i < RT; ++i) wp[i] = w + (int64_t)min(r0 + 16 * i + (lane & 15), R - 1) * K + kb;
  const bf16* xp = x + (int64_t)min(t0 + (lane & 15), T - 1) * ldx + kb;
  f32x4 acc[RT];
#pragma unroll
  for (int i = 0; i < RT; ++i) acc[i] = f32x4{};
  constexpr int U = RT == 1 ? 8 : 4, S = 32 * NW;
  int k = 32 * wid;
  for (; k + S * (U - 1) < K; k += S * U) {
    bf16x8 a[U][RT], b[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      b[u] = *reinterpret_cast<const bf16x8*>(xp + k + S * u);
#pragma unroll
      for (int i = 0; i < RT; ++i) a[u][i] = *reinterpret_cast<const bf16x8*>(wp[i] + k + S * u);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int i = 0; i < RT; ++i) acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[u][i], b[u], acc[i], 0, 0, 0);
  }
  for (; k < K; k += S) {
    const bf16x8 b = *reinterpret_cast<const bf16x8*>(xp + k);
#pragma unroll
    for (int i = 0; i < RT; ++i) {
      const bf16x8 a = *reinterpret_cast<const bf16x8*>(wp[i] + k);
      acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, acc[i], 0, 0, 0);
    }
  }
  if (wid > 0) {
#pragma unroll
    for (int i = 0; i < RT; ++i) red[wid - 1][i][lane] = acc[i];
  }
  __syncthreads();
  if (wid > 0) return;
  const int t = t0 + (lane & 15);
  if (t >= T) return;
#pragma unroll
  for (int i = 0; i < RT; ++i) {
#pragma unroll
    for (int v = 0; v < NW - 1; ++v) acc[i] += red[v][i][lane];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int n = r0 + 16 * i + 4 * (lane >> 4) + r;
      if (n < R) z[(int64_t)t * ldz + n] = acc[i][r];
    }
  }
}

// largest value of the wave and its index (the smaller index among equals); every lane gets both
__device__ __forceinline__ void wave_argmax(float& v, int& i) {
#pragma unroll
  for (int o = 32; o >= 1; o >>= 1) {
    const float ov = __shfl_xor(v, o, 64);
    const int oi = __shfl_xor(i, o, 64);
    if (ov > v || (ov == v && oi < i)) {
      v = ov;
      i = oi;
    }
  }
}

// Entry v of lane l (uniform), for every lane
__device__ __forceinline__ float of_lane(float v, int l) {
  return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), l));
}

// One wave per token; lane l holds entries l + 64 q of the N = experts + identities. groups <= 64. Up to 128 entries every
// lane ranks its own against all others (readlane, no dependent steps); more are picked one by one.
template <int Q>
__global__ __launch_bounds__(256) void router_select_kernel(const float* __restrict__ z, int64_t ldz, int sigmoid,
                                                            const float* __restrict__ correction,
                                                            int* __restrict__ expert, float* __restrict__ weight, int T,
                                                            int N, int groups, int keep, int top, float scale) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (t >= T) return;
  float s[Q], c[Q];
  float m = -INFINITY;
#pragma unroll
  for (int q = 0; q < Q; ++q) {
    const int e = lane + 64 * q;
    s[q] = e < N ? z[(int64_t)t * ldz + e] : -INFINITY;
    m = fmaxf(m, s[q]);
  }
  float inv = 1.f;
  if (sigmoid) {
#pragma unroll
    for (int q = 0; q < Q; ++q) {
      const float e = expf(-fabsf(s[q])), r = 1.f / (1.f + e);
      s[q] = s[q] >= 0.f ? r : e * r;
    }
  } else {
    m = wave_max(m);
    float sum = 0.f;
#pragma unroll
    for (int q = 0; q < Q; ++q) {
      s[q] = lane + 64 * q < N ? expf(s[q] - m) : 0.f;
      sum += s[q];
    }
    inv = 1.f / wave_sum(sum);
  }
#pragma unroll
  for (int q = 0; q < Q; ++q) {
    const int e = lane + 64 * q;
    s[q] *= inv;
    c[q] = e < N ? (correction != nullptr ? s[q] + correction[e] : s[q]) : -INFINITY;
    if (c[q] != c[q]) c[q] = -3.0e38f;  // rank a NaN last: every choice stays a valid index
  }
  if constexpr (Q <= 2) {
    // how many entries go before entry e: greater ones, and equal ones of a smaller index
    auto ranks = [&](int (&rank)[Q]) {
#pragma unroll
      for (int q = 0; q < Q; ++q) rank[q] = 0;
#pragma unroll
      for (int o = 0; o < Q; ++o) {
        // (lanes past the N entries hold -infinity: they come before none of them)
#pragma unroll 16
        for (int l = 0; l < 64; ++l) {
          const float v = of_lane(c[o], l);
#pragma unroll
          for (int q = 0; q < Q; ++q) rank[q] += v > c[q] || (v == c[q] && l + 64 * o < lane + 64 * q);
        }
      }
    };
    int rank[Q];
    if (keep < groups) {
      const int size = N / groups;
      int group[Q], before[Q];
      float best[Q];
#pragma unroll
      for (int q = 0; q < Q; ++q) {
        group[q] = (lane + 64 * q) / size;
        best[q] = -INFINITY;
        before[q] = 0;
      }
      for (int g = 0; g < groups; ++g) {  // group g's largest score: its own entries learn it, all others compare
        float top_g = -INFINITY;
        for (int e = g * size; e < (g + 1) * size; ++e)
          top_g = fmaxf(top_g, of_lane(Q == 2 && e >= 64 ? c[Q - 1] : c[0], e & 63));
#pragma unroll
        for (int q = 0; q < Q; ++q)
          if (group[q] == g) best[q] = top_g;
      }
      for (int g = 0; g < groups; ++g) {
        const int e = g * size;
        const float top_g = of_lane(Q == 2 && e >= 64 ? best[Q - 1] : best[0], e & 63);
#pragma unroll
        for (int q = 0; q < Q; ++q) before[q] += top_g > best[q] || (top_g == best[q] && g < group[q]);
      }
#pragma unroll
      for (int q = 0; q < Q; ++q)
        if (before[q] >= keep) c[q] = -INFINITY;
    }
    ranks(rank);
#pragma unroll
    for (int q = 0; q < Q; ++q)
      if (lane + 64 * q < N && rank[q] < top) {
        expert[(int64_t)t * top + rank[q]] = lane + 64 * q;
        weight[(int64_t)t * top + rank[q]] = s[q] * scale;
      }
    return;
  }
  if (keep < groups) {
    const int size = N / groups;
    float best = -INFINITY;  // lane g: group g's score
    for (int g = 0; g < groups; ++g) {
      float v = -INFINITY;
#pragma unroll
      for (int q = 0; q < Q; ++q) {
        const int e = lane + 64 * q;
        if (e >= g * size && e < (g + 1) * size) v = fmaxf(v, c[q]);
      }
      v = wave_max(v);
      if (lane == g) best = v;
    }
    unsigned long long kept = 0;
    for (int i = 0; i < keep; ++i) {
      float v = best;
      int g = lane;
      wave_argmax(v, g);
      kept |= 1ull << g;
      if (lane == g) best = -INFINITY;
    }
#pragma unroll
    for (int q = 0; q < Q; ++q) {
      const int g = (lane + 64 * q) / size;
      if (g >= groups || !((kept >> g) & 1)) c[q] = -INFINITY;
    }
  }
  for (int j = 0; j < top; ++j) {
    float v = -INFINITY;
    int e = lane;
#pragma unroll
    for (int q = 0; q < Q; ++q)
      if (c[q] > v) {
        v = c[q];
        e = lane + 64 * q;
      }
    wave_argmax(v, e);
    float w = 0.f;
#pragma unroll
    for (int q = 0; q < Q; ++q)
      if (e == lane + 64 * q) {
        c[q] = -INFINITY;
        w = s[q] * scale;
      }
    if (lane == (e & 63)) {
      expert[(int64_t)t * top + j] = e;
      weight[(int64_t)t * top + j] = w;
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------
// choices sorted by expert
// ---------------------------------------------------------------------------------------------------------------
constexpr int kMaxExperts = 1024;

// One workgroup. offs[E + 1]: rows of every expert; row[a] of choice a = token * k + j (identity choices: -1);
// token[row] and, if asked, the choices' weights in the same order; the tile list (expert, first row inside the expert) for products of tm rows.
__global__ __launch_bounds__(1024) void expert_sort_kernel(const int* __restrict__ expert, int n, int k, int E,
                                                           int* __restrict__ offs, int* __restrict__ row,
                                                           int* __restrict__ token, const float* __restrict__ weight,
                                                           float* __restrict__ row_weight, int tm, int* __restrict__ tile_e,
                                                           int* __restrict__ tile_m, int* __restrict__ n_tiles,
                                                           int max_tiles) {
  __shared__ int count[kMaxExperts], start[kMaxExperts], tiles[kMaxExperts], wsum[2][16];
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  count[tid] = 0;
  __syncthreads();
  constexpr int U = 8;  // choices of a thread at a time: their loads and counts overlap
  for (int a0 = tid; a0 < n; a0 += 1024 * U) {
    int e[U], r[U];
#pragma unroll
    for (int u = 0; u < U; ++u) e[u] = a0 + 1024 * u < n ? expert[a0 + 1024 * u] : -1;
#pragma unroll
    for (int u = 0; u < U; ++u) r[u] = e[u] >= 0 && e[u] < E ? atomicAdd(&count[e[u]], 1) : -1;
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (a0 + 1024 * u < n) row[a0 + 1024 * u] = r[u];
  }
  __syncthreads();
  // exclusive sums of the counts and of the tile counts over the experts (thread = expert)
  const int c = tid < E ? count[tid] : 0, tl = (c + tm - 1) / tm;
  int ci = c, ti = tl;
#pragma unroll
  for (int o = 1; o < 64; o <<= 1) {
    const int a = __shfl_up(ci, o, 64), b = __shfl_up(ti, o, 64);
    if (lane >= o) {
      ci += a;
      ti += b;
    }
  }
  if (lane == 63) {
    wsum[0][w] = ci;
    wsum[1][w] = ti;
  }
  __syncthreads();
  for (int i = 0; i < w; ++i) {
    ci += wsum[0][i];
    ti += wsum[1][i];
  }
  start[tid] = ci - c;
  tiles[tid] = ti - tl;
  if (tid < E) offs[tid] = ci - c;
  if (tid == E - 1) {
    offs[E] = ci;
    *n_tiles = min(ti, max_tiles);
  }
  __syncthreads();
  for (int e = w; e < E; e += 16) {
    const int nt = (count[e] + tm - 1) / tm;
    for (int i = lane; i < nt; i += 64) {
      const int at = tiles[e] + i;
      if (at < max_tiles) {
        tile_e[at] = e;
        tile_m[at] = i * tm;
      }
    }
  }
  for (int a0 = tid; a0 < n; a0 += 1024 * U) {
    int e[U], r[U];
    float wt[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int a = min(a0 + 1024 * u, n - 1);
      e[u] = expert[a];
      r[u] = row[a];  // written by this thread above
      wt[u] = row_weight != nullptr ? weight[a] : 0.f;
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int a = a0 + 1024 * u;
      if (a >= n || r[u] < 0) continue;
      row[a] = start[e[u]] + r[u];
      token[start[e[u]] + r[u]] = a / k;
      if (row_weight != nullptr) row_weight[start[e[u]] + r[u]] = wt[u];
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------
// products of few rows, straight from the choices
// ---------------------------------------------------------------------------------------------------------------
// out[a] = act(x[a / kx] . Wg[e]^T) * (x[a / kx] . Wu[e]^T) (GLU) or x[a / kx] . W[e]^T, for every choice a of expert e;
// W of expert e is [rows, K] with rows = 2N (GLU: gate rows, then up rows) or N. Behind the routed slots, n_sh tokens
// through the shared expert. A workgroup: one expert and 16 output columns; its four waves split K and hold the
// weights of one pass over up to 16 rows each (mfma_f32_16x16x32_bf16, A = weights, B = rows), as in gemv.hip.
struct SkinnyParams {
  const bf16* x;
  int64_t ldx;
  const bf16* w;       // [E, rows, K]
  bf16* out;           // [n, ldo]
  int64_t ldo;
  const int* expert;   // [n]
  int n, kx, E, N, K, slots;
  const bf16* xs;      // shared expert
  int64_t ldxs;
  const bf16* ws;      // [rows, Ks] or null
  bf16* outs;          // [n_sh, ldos]
  int64_t ldos;
  int n_sh, Ns, Ks;
  int act;             // GLU: 0 silu, 5 the clamped unit
  float limit;
  const float* weight; // [n] or null: GLU multiplies the routed rows' products with it
};

__device__ __forceinline__ float gated_unit(float g, float u, int act, float limit) {
  if (act == 0) return g / (1.f + __expf(-g)) * u;
  g = fminf(g, limit);
  return g / (1.f + __expf(-1.702f * g)) * (fminf(fmaxf(u, -limit), limit) + 1.f);
}

constexpr int kSkinnyMax = 2048;  // choices

template <bool GLU>
__global__ __launch_bounds__(256) void experts_skinny_kernel(SkinnyParams p) {
  constexpr int R = GLU ? 2 : 1;
  __shared__ f32x4 red[3][R][64];
  __shared__ int list[kSkinnyMax];
  __shared__ int s_n;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int nt = (p.N + 15) / 16;
  int id = blockIdx.x;
  const bf16 *x, *w;
  bf16* out;
  int64_t ldx, ldo;
  int N, K, rows, kx;
  const bool routed = id < p.slots * nt;
  if (routed) {
    const int slot = id / nt;
    id -= slot * nt;
    // with fewer choices than experts a slot is a choice, and the first choice of an expert serves all of them
    const int e = p.slots == p.n ? p.expert[slot] : slot;
    if (e < 0 || e >= p.E) return;
    if (threadIdx.x == 0) s_n = 0;
    __syncthreads();
    for (int a0 = 0; a0 < p.n; a0 += 256) {
      const int a = a0 + threadIdx.x;
      if (a < p.n && p.expert[a] == e) list[atomicAdd(&s_n, 1)] = a;
    }
    __syncthreads();
    rows = s_n;
    if (rows == 0) return;
    if (p.slots == p.n) {
      int first = list[0];
      for (int i = 1; i < rows; ++i) first = min(first, list[i]);
      if (first != slot) return;
    }
    x = p.x; ldx = p.ldx; kx = p.kx; out = p.out; ldo = p.ldo; N = p.N; K = p.K;
    w = p.w + (int64_t)e * (R * N) * K;
  } else {
    id -= p.slots * nt;
    rows = p.n_sh;
    x = p.xs; ldx = p.ldxs; kx = 1; out = p.outs; ldo = p.ldos; N = p.Ns; K = p.Ks;
    w = p.ws;
  }
  const int n0 = id * 16;
  const int kq = K >> 2, kb = wid * kq + 8 * (lane >> 4);
  const bf16* wp[R];
#pragma unroll
  for (int r = 0; r < R; ++r) wp[r] = w + ((int64_t)r * N + min(n0 + (lane & 15), N - 1)) * K + kb;
  for (int g = 0; g < rows; g += 16) {
    const int i = g + (lane & 15);
    const bool ok = i < rows;
    const int a = routed ? list[ok ? i : rows - 1] : (ok ? i : rows - 1);
    const bf16* xp = x + (int64_t)(a / kx) * ldx + kb;
    f32x4 acc[R];
#pragma unroll
    for (int r = 0; r < R; ++r) acc[r] = f32x4{};
    constexpr int U = GLU ? 8 : 8;
    int k = 0;
    for (; k + 32 * U <= kq; k += 32 * U) {
      bf16x8 wv[U][R], xv[U];
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int r = 0; r < R; ++r) wv[u][r] = *reinterpret_cast<const bf16x8*>(wp[r] + k + 32 * u);
#pragma unroll
      for (int u = 0; u < U; ++u) xv[u] = *reinterpret_cast<const bf16x8*>(xp + k + 32 * u);
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int r = 0; r < R; ++r)
          acc[r] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv[u][r], xv[u], acc[r], 0, 0, 0);
    }
    for (; k < kq; k += 32) {
      const bf16x8 xv = *reinterpret_cast<const bf16x8*>(xp + k);
#pragma unroll
      for (int r = 0; r < R; ++r)
        acc[r] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(wp[r] + k), xv, acc[r], 0, 0,
                                                         0);
    }
    if (g > 0) __syncthreads();  // the previous rows' partial sums have been read
    if (wid > 0) {
#pragma unroll
      for (int r = 0; r < R; ++r) red[wid - 1][r][lane] = acc[r];
    }
    __syncthreads();
    if (wid == 0 && ok) {
#pragma unroll
      for (int r = 0; r < R; ++r)
#pragma unroll
        for (int v = 0; v < 3; ++v) acc[r] += red[v][r][lane];
      const float rw = GLU && routed && p.weight != nullptr ? p.weight[a] : 1.f;
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const int n = n0 + 4 * (lane >> 4) + q;
        float v = acc[0][q];
        if constexpr (GLU) v = gated_unit(v * rw, acc[R - 1][q] * rw, p.act, p.limit);
        if (n < N) out[(int64_t)a * ldo + n] = (bf16)v;
      }
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------
// 32-bit grouped product: y[rows of e] = x[...] . w[e]^T, any sizes; 64 x 64 tiles, 4 x 4 outputs per thread
// ---------------------------------------------------------------------------------------------------------------
__global__ __launch_bounds__(256) void experts_gemm_f32_kernel(const float* __restrict__ x, int64_t ldx,
                                                               const float* __restrict__ w, float* __restrict__ y,
                                                               int64_t ldy, const int* __restrict__ src,
                                                               const int* __restrict__ offs,
                                                               const int* __restrict__ tile_e,
                                                               const int* __restrict__ tile_m,
                                                               const int* __restrict__ n_tiles,
                                                               const float* __restrict__ row_weight, int rows_max, int N,
                                                               int K) {
  const int t = blockIdx.y;
  if (t >= *n_tiles) return;
  __shared__ float sx[16][65], sw[16][65];
  const int e = tile_e[t], r0 = offs[e] + tile_m[t], r1 = min(offs[e + 1], rows_max), n0 = blockIdx.x * 64;
  const float* we = w + (int64_t)e * N * K;
  const int tx = threadIdx.x & 15, ty = threadIdx.x >> 4;
  const int lr = threadIdx.x >> 2, lk = (threadIdx.x & 3) * 4;
  const int xr = min(r0 + lr, r1 - 1);
  const float* xp = x + (int64_t)(src != nullptr ? src[xr] : xr) * ldx;
  const float* wp = we + (int64_t)min(n0 + lr, N - 1) * K;
  float acc[4][4] = {};
  for (int k0 = 0; k0 < K; k0 += 16) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int k = k0 + lk + i;
      sx[lk + i][lr] = k < K ? xp[k] : 0.f;
      sw[lk + i][lr] = k < K ? wp[k] : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < 16; ++k) {
      float a[4], b[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        a[i] = sx[k][ty * 4 + i];
        b[i] = sw[k][tx * 4 + i];
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] += a[i] * b[j];
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = r0 + ty * 4 + i;
    if (r >= r1) continue;
    const float rw = row_weight != nullptr ? row_weight[r] : 1.f;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int n = n0 + tx * 4 + j;
      if (n < N) y[(int64_t)r * ldy + n] = acc[i][j] * rw;
    }
  }
}

}  // namespace

// bf16 x [T, ldx] and w [R, K]; z [T, ldz]. K % 128 == 0, 16-B rows.
HDS_EXPORT int hds_router_logits(const void* x, int64_t ldx, const void* w, float* z, int64_t ldz, int T, int R, int K,
                                 hipStream_t st) {
  if (T <= 0) return 0;
  if (R < 1 || K < 128 || K % 128 || ldx % 8 || ldx < K || ldz < R) return hipErrorInvalidValue;
#define HDS_RL(RT, NW)                                                                                               \
  hipLaunchKernelGGL((router_logits_kernel<RT, NW>), dim3((R + 16 * RT - 1) / (16 * RT), (T + 15) / 16),            \
                     dim3(64 * NW), 0, st, (const bf16*)x, ldx, (const bf16*)w, z, ldz, T, R, K)
  if (T >= 512) HDS_RL(5, 8); else if (T > 64) HDS_RL(1, 4); else HDS_RL(1, 16);
#undef HDS_RL
  return hipGetLastError();
}

// N = experts + identities <= 1024, in `groups` <= 64 equal groups of which `keep` take part; sigmoid: scores are sigmoid(z),
// not softmax(z); correction may be null
HDS_EXPORT int hds_router_select(const float* z, int64_t ldz, int sigmoid, const float* correction, int* expert, float* weight,
                                 int T, int N, int groups, int keep, int top, float scale, hipStream_t st) {
  if (T <= 0) return 0;
  if (N < 1 || N > 1024 || ldz < N || groups < 1 || groups > 64 || N % groups || keep < 1 || keep > groups || top < 1 ||
      top > keep * (N / groups))
    return hipErrorInvalidValue;
#define HDS_RS(Q)                                                                                                   \
  hipLaunchKernelGGL(router_select_kernel<Q>, dim3((T + 3) / 4), dim3(256), 0, st, z, ldz, sigmoid, correction, expert, \
                     weight, T, N, groups, keep, top, scale)
  if (N <= 64) HDS_RS(1); else if (N <= 128) HDS_RS(2); else if (N <= 256) HDS_RS(4); else if (N <= 512) HDS_RS(8);
  else HDS_RS(16);
#undef HDS_RS
  return hipGetLastError();
}

// n = tokens * k choices; row [n], token [n], weight and row_weight [n] or null, offs [E + 1], tile lists of max_tiles >= n / tm + E entries
HDS_EXPORT int hds_expert_sort(const int* expert, int n, int k, int E, int* offs, int* row, int* token,
                               const float* weight, float* row_weight, int tm,
                               int* tile_e, int* tile_m, int* n_tiles, int max_tiles, hipStream_t st) {
  if (n <= 0) return 0;
  if (k < 1 || E < 1 || E > kMaxExperts || tm < 1 || (row_weight != nullptr && weight == nullptr) || max_tiles < n / tm + (E < n ? E : n)) return hipErrorInvalidValue;
  hipLaunchKernelGGL(expert_sort_kernel, dim3(1), dim3(1024), 0, st, expert, n, k, E, offs, row, token, weight,
                     row_weight, tm, tile_e,
                     tile_m, n_tiles, max_tiles);
  return hipGetLastError();
}

HDS_EXPORT int hds_experts_skinny_max() { return kSkinnyMax; }

// See SkinnyParams. glu: w / ws hold gate and up rows, act 0 (silu) or 5 (clamped, with limit). kx: choices per row of x. K, Ks % 128 == 0; 16-B rows.
HDS_EXPORT int hds_experts_skinny(int glu, const void* x, int64_t ldx, const void* w, void* out, int64_t ldo,
                                  const int* expert, int n, int kx, int E, int N, int K, const void* xs, int64_t ldxs,
                                  const void* ws, void* outs, int64_t ldos, int n_sh, int Ns, int Ks, int act,
                                  float limit, const float* weight, hipStream_t st) {
  if (n <= 0) return 0;
  const bool sh = ws != nullptr && n_sh > 0;
  if (n > kSkinnyMax || (act != 0 && act != 5) || kx < 1 || E < 1 || N < 1 || K < 128 || K % 128 || ldx < K || ldx % 8 || ldo < N ||
      (sh && (Ns < 1 || Ks < 128 || Ks % 128 || ldxs < Ks || ldxs % 8 || ldos < Ns)))
    return hipErrorInvalidValue;
  const int slots = n < E ? n : E;
  // n == E: a slot may be read as a choice or as an expert; both cover everything once
  SkinnyParams p{(const bf16*)x, ldx, (const bf16*)w, (bf16*)out, ldo, expert, n, kx, E, N, K, slots, (const bf16*)xs,
                 ldxs, (const bf16*)ws, (bf16*)outs, ldos, sh ? n_sh : 0, Ns, Ks, act, limit, weight};
  const int64_t blocks = (int64_t)slots * ((N + 15) / 16) + (sh ? (Ns + 15) / 16 : 0);
  if (glu)
    hipLaunchKernelGGL(experts_skinny_kernel<true>, dim3(blocks), dim3(256), 0, st, p);
  else
    hipLaunchKernelGGL(experts_skinny_kernel<false>, dim3(blocks), dim3(256), 0, st, p);
  return hipGetLastError();
}

// rows of 64-row tiles (expert_sort with tm = 64); src: row of x for every sorted row (null: the row itself);
// row_weight [rows] or null multiplies the results
HDS_EXPORT int hds_experts_gemm_f32(const float* x, int64_t ldx, const float* w, float* y, int64_t ldy, const int* src,
                                    const int* offs, const int* tile_e, const int* tile_m, const int* n_tiles,
                                    int max_tiles, const float* row_weight, int rows, int N, int K, hipStream_t st) {
  if (rows <= 0) return 0;
  if (N < 1 || K < 1 || ldx < K || ldy < N || max_tiles < 1 || max_tiles > 65535) return hipErrorInvalidValue;
  hipLaunchKernelGGL(experts_gemm_f32_kernel, dim3((N + 63) / 64, max_tiles), dim3(256), 0, st, x, ldx, w, y, ldy, src,
                     offs, tile_e, tile_m, n_tiles, row_weight, rows, N, K);
  return hipGetLastError();
}
