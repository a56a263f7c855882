// Latent (compressed K/V) attention over a paged cache. A cached row holds, for one token and all heads, the normed
// latent c [rank] and one rotated key part r [rot]: heads share it, per head k = W_uk[h] c (unrotated part), v = W_uv[h] c.
//
//   score(i, j, h) = scale * (q_nope[i, h] . W_uk[h] c_j + q_rot[i, h] . r_j),  0 <= i - j < window (0: no window)
//
// and optionally a gate per token and head whose sigmoid multiplies the head's output.
//
// Two forms of the same product, chosen per sequence of a step:
//   * absorbed (single tokens, short portions): W_uk[h]^T q_nope is formed once per token and head, scores and the
//     weighted sum run on the cached rows themselves (read once for all heads), W_uv[h] is applied to the sum;
//   * expanded (prompt portions): the visible rows are gathered, k and v of all heads come from one matrix product,
//     and an MFMA flash kernel runs over them.
//
// Kernels: latent_prep (norm of c, rotation of the shared key part and of q, cache scatter, absorption of W_uk),
// latent_decode (absorbed, split over keys; MFMA in
// bf16, a plain kernel for 32-bit and odd sizes), latent_combine (merges the splits, applies W_uv), latent_prefill.
#include "attn_common.h"

using namespace hds;
using namespace hds::attn;

namespace {

constexpr float kLog2e = 1.4426950408889634f;

__device__ __forceinline__ float gate_of(float g) { return 1.f / (1.f + __expf(-g)); }

template <typename T>
struct PrepParams {
  T* q;                   // [tokens, ldq]: per head [dim | rot]
  int64_t ldq;
  const T* c;             // [tokens, ldc]: latent [rank], then the shared key part [rot]
  int64_t ldc;
  const float* norm;      // [rank]
  const float* cos_t;     // [positions, rd / 2]
  const float* sin_t;
  T* cache;               // pages of [block_size, rank + rot]
  const int* tok_seq;
  const int* tok_pos;
  const int* tables;
  const int* ws_row;      // [tokens] row of ws for expanded tokens, -1: none; null: none
  T* ws;                  // [rows, rank + rot]
  const T* uk;            // [H, dim, rank]
  const int* atok;        // [n_abs] token of every absorbed row; null: row a is token a
  T* qa;                  // [n_abs, H, rank + rot]
  int n_tok, n_abs, n_pos, max_blocks, block_size, H, dim, rot, rdims, rank;
  float eps;
};

// interleaved rotation: (2i, 2i+1) turn together for i < rdims / 2, the rest of the rot part passes
template <typename T>
__device__ __forceinline__ float rotated(const T* v, int e, int rdims, const float* c, const float* s) {
  const float x = to_f(v[e]);
  if (e >= rdims) return x;
  const float y = to_f(v[e ^ 1]);
  const float cc = c[e >> 1], ss = s[e >> 1];
  return (e & 1) ? x * cc + y * ss : x * cc - y * ss;
}

// 8 elements e .. e + 7 of a rotated part (rdims and e multiples of 8)
template <typename T>
__device__ __forceinline__ void rotate8(float (&v)[8], int e, int rdims, const float* c, const float* s) {
  if (e >= rdims) return;
  const f32x4 cc = *reinterpret_cast<const f32x4*>(c + e / 2), sn = *reinterpret_cast<const f32x4*>(s + e / 2);
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    const float a = v[2 * k], b = v[2 * k + 1];
    v[2 * k] = a * cc[k] - b * sn[k];
    v[2 * k + 1] = b * cc[k] + a * sn[k];
  }
}

constexpr int kAbsTok = 4;    // absorbed tokens that share one read of W_uk[h]
constexpr int kAbsCols = 128; // latent columns of an absorption workgroup (vector path)

// Vector path (all part sizes multiples of 8, rank <= 2048). Workgroups [0, n_tok): one token each (norm, rotation,
// scatter, q of expanded tokens rotated in place); then one per (head, kAbsCols columns, TG absorbed tokens).
// TG: absorbed tokens a workgroup takes; 0: none in the batch.
template <typename T, int TG>
__global__ __launch_bounds__(256) void latent_prep8_kernel(PrepParams<T> p) {
  extern __shared__ float sm[];
  const int qh = p.dim + p.rot, row_w = p.rank + p.rot;
  const int half = p.rdims / 2;
  if ((int)blockIdx.x < p.n_tok) {
    const int t = blockIdx.x;
    const int pos = min(p.tok_pos[t], p.n_pos - 1);
    const float* ct = p.cos_t + (int64_t)pos * half;
    const float* st = p.sin_t + (int64_t)pos * half;
    T* row = p.q + (int64_t)t * p.ldq;
    const T* c = p.c + (int64_t)t * p.ldc;
    const int nc = row_w / 8;
    const int i = threadIdx.x;  // chunk of the row; rows of more than 256 chunks loop below for the rotated part only
    float v[8];
    float ss = 0.f;
    if (8 * i < p.rank) {
      Vec8<T>::load(c + 8 * i, v);
#pragma unroll
      for (int k = 0; k < 8; ++k) ss += v[k] * v[k];
    }
    const int blk = p.tables[(int64_t)p.tok_seq[t] * p.max_blocks + pos / p.block_size];
    T* dst = p.cache + ((int64_t)blk * p.block_size + pos % p.block_size) * row_w;
    const int wr = p.ws_row != nullptr ? p.ws_row[t] : -1;
    T* dst2 = wr >= 0 ? p.ws + (int64_t)wr * row_w : nullptr;
    if (wr >= 0) {
      const int nq = p.rdims / 8;
      for (int q = threadIdx.x; q < p.H * nq; q += 256) {
        const int h = q / nq, e = 8 * (q - h * nq);
        T* a = row + (int64_t)h * qh + p.dim + e;
        float x[8];
        Vec8<T>::load(a, x);
        rotate8<T>(x, e, p.rdims, ct, st);
        Vec8<T>::store(a, x);
      }
    }
    ss = block_sum<256>(ss, sm);
    const float rs = 1.f / sqrtf(ss / (float)p.rank + p.eps);
    if (8 * i < p.rank) {
      float n[8];
      Vec8<float>::load(p.norm + 8 * i, n);
#pragma unroll
      for (int k = 0; k < 8; ++k) v[k] *= rs * n[k];
      Vec8<T>::store(dst + 8 * i, v);
      if (dst2 != nullptr) Vec8<T>::store(dst2 + 8 * i, v);
    }
    for (int j = p.rank / 8 + threadIdx.x; j < nc; j += 256) {
      Vec8<T>::load(c + 8 * j, v);
      rotate8<T>(v, 8 * j - p.rank, p.rdims, ct, st);
      Vec8<T>::store(dst + 8 * j, v);
      if (dst2 != nullptr) Vec8<T>::store(dst2 + 8 * j, v);
    }
    return;
  }
  if constexpr (TG > 0) {
    const int ncb = (p.rank + kAbsCols - 1) / kAbsCols;
    int w = blockIdx.x - p.n_tok;
    const int h = w % p.H;
    w /= p.H;
    const int cb = w % ncb, a0 = (w / ncb) * TG;
    const int na = min(TG, p.n_abs - a0);
    float* sq = sm;                    // [TG][dim]
    float* red = sm + TG * p.dim;      // [4 waves][TG][kAbsCols]
    // 16 lanes cover the columns, the 16 lane groups of the workgroup take every 16th row of W_uk[h]
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int col = cb * kAbsCols + 8 * (lane & 15), dg = wid * 4 + (lane >> 4);
    const T* uk = p.uk + (int64_t)h * p.dim * p.rank + (col < p.rank ? col : 0);
    float u[8][8];
    auto fetch = [&](int d0) {
#pragma unroll
      for (int b = 0; b < 8; ++b)
        if (d0 + 16 * b < p.dim) Vec8<T>::load(uk + (int64_t)(d0 + 16 * b) * p.rank, u[b]);
    };
    fetch(dg);
    for (int i = threadIdx.x; i < TG * p.dim; i += 256) {
      const int a = i / p.dim, d = i - a * p.dim;
      float v = 0.f;
      if (a < na) {
        const int t = p.atok != nullptr ? p.atok[a0 + a] : a0 + a;
        v = to_f(p.q[(int64_t)t * p.ldq + (int64_t)h * qh + d]);
      }
      sq[i] = v;
    }
    if (cb == 0) {
      const int nr = p.rot / 8;
      for (int i = threadIdx.x; i < na * nr; i += 256) {
        const int a = i / nr, e = 8 * (i - a * nr);
        const int t = p.atok != nullptr ? p.atok[a0 + a] : a0 + a;
        const int pos = min(p.tok_pos[t], p.n_pos - 1);
        float x[8];
        Vec8<T>::load(p.q + (int64_t)t * p.ldq + (int64_t)h * qh + p.dim + e, x);
        rotate8<T>(x, e, p.rdims, p.cos_t + (int64_t)pos * half, p.sin_t + (int64_t)pos * half);
        Vec8<T>::store(p.qa + ((int64_t)(a0 + a) * p.H + h) * row_w + p.rank + e, x);
      }
    }
    float acc[TG][8];
#pragma unroll
    for (int a = 0; a < TG; ++a)
#pragma unroll
      for (int k = 0; k < 8; ++k) acc[a][k] = 0.f;
    __syncthreads();
    for (int d0 = dg; d0 < p.dim; d0 += 128) {
      if (d0 != dg) fetch(d0);
#pragma unroll
      for (int b = 0; b < 8; ++b) {
        const int d = d0 + 16 * b;
        if (d >= p.dim) break;
#pragma unroll
        for (int a = 0; a < TG; ++a) {
          const float q = sq[a * p.dim + d];
#pragma unroll
          for (int k = 0; k < 8; ++k) acc[a][k] += q * u[b][k];
        }
      }
    }
#pragma unroll
    for (int a = 0; a < TG; ++a)
#pragma unroll
      for (int k = 0; k < 8; ++k) {
        float v = acc[a][k];
        v += __shfl_xor(v, 16, 64);
        v += __shfl_xor(v, 32, 64);
        if (lane < 16) red[(wid * TG + a) * kAbsCols + 8 * lane + k] = v;
      }
    __syncthreads();
    for (int i = threadIdx.x; i < na * kAbsCols; i += 256) {
      const int a = i / kAbsCols, cc = i - a * kAbsCols;
      if (cb * kAbsCols + cc >= p.rank) continue;
      float v = 0.f;
#pragma unroll
      for (int x = 0; x < 4; ++x) v += red[(x * TG + a) * kAbsCols + cc];
      p.qa[((int64_t)(a0 + a) * p.H + h) * row_w + cb * kAbsCols + cc] = from_f<T>(v);
    }
  }
}

// any sizes; workgroups [0, n_tok): one token each, then ceil(n_abs / kAbsTok) x H: absorption
template <typename T>
__global__ __launch_bounds__(256) void latent_prep_kernel(PrepParams<T> p) {
  extern __shared__ float sm[];
  const int qh = p.dim + p.rot, row_w = p.rank + p.rot;
  if ((int)blockIdx.x < p.n_tok) {
    const int t = blockIdx.x;
    const int pos = min(p.tok_pos[t], p.n_pos - 1);
    const float* ct = p.cos_t + (int64_t)pos * (p.rdims / 2);
    const float* st = p.sin_t + (int64_t)pos * (p.rdims / 2);
    T* row = p.q + (int64_t)t * p.ldq;
    const T* c = p.c + (int64_t)t * p.ldc;
    float ss = 0.f;
    for (int i = threadIdx.x; i < p.rank; i += 256) {
      const float v = to_f(c[i]);
      ss += v * v;
    }
    ss = block_sum<256>(ss, sm);
    const float rs = 1.f / sqrtf(ss / (float)p.rank + p.eps);
    const int blk = p.tables[(int64_t)p.tok_seq[t] * p.max_blocks + pos / p.block_size];
    T* dst = p.cache + ((int64_t)blk * p.block_size + pos % p.block_size) * row_w;
    const int wr = p.ws_row != nullptr ? p.ws_row[t] : -1;
    T* dst2 = wr >= 0 ? p.ws + (int64_t)wr * row_w : nullptr;
    for (int i = threadIdx.x; i < row_w; i += 256) {
      const float v = i < p.rank ? to_f(c[i]) * rs * p.norm[i] : rotated(c + p.rank, i - p.rank, p.rdims, ct, st);
      const T o = from_f<T>(v);
      dst[i] = o;
      if (dst2 != nullptr) dst2[i] = o;
    }
    if (wr >= 0) {
      for (int i = threadIdx.x; i < p.H * (p.rdims / 2); i += 256) {
        const int h = i / (p.rdims / 2), e = 2 * (i - h * (p.rdims / 2));
        T* v = row + (int64_t)h * qh + p.dim;
        const float a = rotated(v, e, p.rdims, ct, st), b = rotated(v, e + 1, p.rdims, ct, st);
        v[e] = from_f<T>(a);
        v[e + 1] = from_f<T>(b);
      }
    }
    return;
  }
  const int w = blockIdx.x - p.n_tok;
  const int h = w % p.H, a0 = (w / p.H) * kAbsTok;
  const int na = min(kAbsTok, p.n_abs - a0);
  for (int i = threadIdx.x; i < na * p.dim; i += 256) {
    const int a = i / p.dim, d = i - a * p.dim;
    const int t = p.atok != nullptr ? p.atok[a0 + a] : a0 + a;
    sm[i] = to_f(p.q[(int64_t)t * p.ldq + (int64_t)h * qh + d]);
  }
  for (int i = na * p.dim + threadIdx.x; i < kAbsTok * p.dim; i += 256) sm[i] = 0.f;
  __syncthreads();
  const T* uk = p.uk + (int64_t)h * p.dim * p.rank;
  for (int i = threadIdx.x; i < p.rank; i += 256) {
    float acc[kAbsTok];
#pragma unroll
    for (int a = 0; a < kAbsTok; ++a) acc[a] = 0.f;
    int d = 0;
    for (; d + 8 <= p.dim; d += 8) {
      float u[8];
#pragma unroll
      for (int k = 0; k < 8; ++k) u[k] = to_f(uk[(int64_t)(d + k) * p.rank + i]);
#pragma unroll
      for (int k = 0; k < 8; ++k)
#pragma unroll
        for (int a = 0; a < kAbsTok; ++a) acc[a] += u[k] * sm[a * p.dim + d + k];
    }
    for (; d < p.dim; ++d) {
      const float u = to_f(uk[(int64_t)d * p.rank + i]);
#pragma unroll
      for (int a = 0; a < kAbsTok; ++a) acc[a] += u * sm[a * p.dim + d];
    }
#pragma unroll
    for (int a = 0; a < kAbsTok; ++a)
      if (a < na) p.qa[((int64_t)(a0 + a) * p.H + h) * row_w + i] = from_f<T>(acc[a]);
  }
  for (int i = threadIdx.x; i < na * p.rot; i += 256) {
    const int a = i / p.rot, e = i - a * p.rot;
    const int t = p.atok != nullptr ? p.atok[a0 + a] : a0 + a;
    const int pos = min(p.tok_pos[t], p.n_pos - 1);
    const T* v = p.q + (int64_t)t * p.ldq + (int64_t)h * qh + p.dim;
    p.qa[((int64_t)(a0 + a) * p.H + h) * row_w + p.rank + e] =
        from_f<T>(rotated(v, e, p.rdims, p.cos_t + (int64_t)pos * (p.rdims / 2), p.sin_t + (int64_t)pos * (p.rdims / 2)));
  }
}

// ---------------------------------------------------------------------------------------------------------------
// absorbed form
// ---------------------------------------------------------------------------------------------------------------
template <typename T>
struct DecodeParams {
  const T* qa;      // [n_abs, H, rank + rot]
  const T* cache;
  float* part_o;    // [n_abs, H, splits, rank], not divided by the sum
  float* part_ml;   // [n_abs, H, splits, 2] max (natural log domain) and sum
  const int* atok;
  const int* tok_seq;
  const int* tok_pos;
  const int* tables;
  int max_blocks, block_size, H, rank, rot, splits, window;
  float scale;
};

template <typename T>
__device__ __forceinline__ void key_range(const DecodeParams<T>& p, int t, int split, int& j0, int& j1) {
  const int pos = p.tok_pos[t];
  const int lo = p.window > 0 ? max(0, pos - p.window + 1) : 0;
  const int n = pos + 1 - lo;
  const int per = (n + p.splits - 1) / p.splits;
  j0 = lo + split * per;
  j1 = min(pos + 1, j0 + per);
}

constexpr int kGenKeys = 64;

// any type and size: one workgroup per (split, head, absorbed row); a wave's lanes share the dims of a key, then every
// thread owns latent columns
template <typename T>
__global__ __launch_bounds__(256) void latent_decode_plain_kernel(DecodeParams<T> p) {
  extern __shared__ float sm[];  // q [rank + rot], scores [kGenKeys], acc [rank]
  const int row_w = p.rank + p.rot;
  float* sq = sm;
  float* ss = sm + row_w;
  float* acc = ss + kGenKeys;
  const int split = blockIdx.x, h = blockIdx.y, a = blockIdx.z;
  const int t = p.atok != nullptr ? p.atok[a] : a;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  int j0, j1;
  key_range(p, t, split, j0, j1);
  const int* table = p.tables + (int64_t)p.tok_seq[t] * p.max_blocks;
  for (int i = threadIdx.x; i < row_w; i += 256) sq[i] = to_f(p.qa[((int64_t)a * p.H + h) * row_w + i]);
  for (int i = threadIdx.x; i < p.rank; i += 256) acc[i] = 0.f;
  __syncthreads();
  auto rowp = [&](int j) {
    return p.cache + ((int64_t)table[j / p.block_size] * p.block_size + j % p.block_size) * row_w;
  };
  float m = -INFINITY, l = 0.f;
  for (int jb = j0; jb < j1; jb += kGenKeys) {
    const int nk = min(kGenKeys, j1 - jb);
    for (int k = w; k < nk; k += 4) {
      const T* kr = rowp(jb + k);
      float s = 0.f;
      for (int i = lane; i < row_w; i += 64) s += sq[i] * to_f(kr[i]);
      s = wave_sum(s);
      if (lane == 0) ss[k] = s * p.scale;
    }
    __syncthreads();
    float mt = m;
    for (int k = 0; k < nk; ++k) mt = fmaxf(mt, ss[k]);
    const float alpha = __expf(m - mt);  // 0 at the first tile
    m = mt;
    float sum = 0.f;
    for (int k = 0; k < nk; ++k) sum += __expf(ss[k] - m);
    l = l * alpha + sum;
    for (int i = threadIdx.x; i < p.rank; i += 256) {
      float o = acc[i] * alpha;
      for (int k = 0; k < nk; ++k) o += __expf(ss[k] - m) * to_f(rowp(jb + k)[i]);
      acc[i] = o;
    }
    __syncthreads();
  }
  const int64_t pi = ((int64_t)a * p.H + h) * p.splits + split;
  for (int i = threadIdx.x; i < p.rank; i += 256) p.part_o[pi * p.rank + i] = acc[i];
  if (threadIdx.x == 0) {
    p.part_ml[2 * pi] = m;
    p.part_ml[2 * pi + 1] = l;
  }
}

// bf16, rank and rot multiples of 8: 16 HG heads of one absorbed row on the matrix cores, 64 keys a tile. The key tile
// is one LDS image read by rows for the scores (A = keys, B = q: the accumulator column is the head) and transposed for
// the weighted sum (A = weights, B = latent columns). Four waves per group of 16 heads: each takes 16 keys of the
// scores, then every fourth 16-column block of the latent (NB of them at most). A thread stages NCH 16-byte chunks of
// one key row and requests the next tile's before it computes on this one.
constexpr int kTK = 64;

template <int HG, int NCH, int NB>
__global__ __launch_bounds__(256 * HG) void latent_decode_mfma_kernel(DecodeParams<bf16> p) {
  extern __shared__ __attribute__((aligned(16))) char lds[];
  constexpr int NT = 256 * HG, TPR = 4 * HG;    // threads; of them on one key row
  const int row_w = p.rank + p.rot;
  const int kd = (row_w + 31) & ~31;            // contraction length, zero padded
  const int ldk = kd + 8;                       // LDS row stride (elements)
  bf16* sk = reinterpret_cast<bf16*>(lds);      // [kTK][ldk]
  bf16* sq = sk + kTK * ldk;                    // [16 HG][ldk]
  const int lane = threadIdx.x & 63, hg = threadIdx.x >> 8, w = (threadIdx.x >> 6) & 3;
  bf16* sp = sq + 16 * HG * ldk + hg * 16 * (kTK + 8);  // [HG][16][kTK + 8]
  float* smax = reinterpret_cast<float*>(sq + 16 * HG * ldk + HG * 16 * (kTK + 8)) + hg * 128;  // [HG][4][16]
  float* ssum = smax + 64;                              // [HG][4][16]
  const int split = blockIdx.x, hb = blockIdx.y * 16 * HG, a = blockIdx.z;
  const int h0 = hb + 16 * hg;
  const int t = p.atok != nullptr ? p.atok[a] : a;
  const int l15 = lane & 15, g = lane >> 4;
  int j0, j1;
  key_range(p, t, split, j0, j1);
  const int* table = p.tables + (int64_t)p.tok_seq[t] * p.max_blocks;
  const int nch = row_w / 8, nchp = kd / 8;
  const bf16x8 zero = {};
  const int kr = threadIdx.x / TPR, kc = threadIdx.x % TPR;
  bf16x8 pf[NCH];
  auto fetch = [&](int jb) {
    const int j = jb + kr;
    const bool ok = j < j1;
    const bf16* src = p.cache;
    if (ok) src += ((int64_t)table[j / p.block_size] * p.block_size + j % p.block_size) * row_w;
#pragma unroll
    for (int k = 0; k < NCH; ++k) {
      const int c = kc + TPR * k;
      pf[k] = zero;
      if (ok && c < nch) pf[k] = *reinterpret_cast<const bf16x8*>(src + 8 * c);
    }
  };
  if (j0 < j1) fetch(j0);
  for (int i = threadIdx.x; i < 16 * HG * nchp; i += NT) {
    const int r = i / nchp, c = i - r * nchp;
    bf16x8 v = zero;
    if (hb + r < p.H && c < nch)
      v = *reinterpret_cast<const bf16x8*>(p.qa + ((int64_t)a * p.H + hb + r) * row_w + 8 * c);
    *reinterpret_cast<bf16x8*>(sq + r * ldk + 8 * c) = v;
  }
  f32x4 o[NB];
#pragma unroll
  for (int b = 0; b < NB; ++b) o[b] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;  // of head l15 (replicated over the lane groups and the head group's waves)
  const float c2 = p.scale * kLog2e;
  for (int jb = j0; jb < j1; jb += kTK) {
    if (jb > j0) __syncthreads();  // the previous tile is read out
#pragma unroll
    for (int k = 0; k < NCH; ++k) {
      const int c = kc + TPR * k;
      if (c < nchp) *reinterpret_cast<bf16x8*>(sk + kr * ldk + 8 * c) = pf[k];
    }
    __syncthreads();
    if (jb + kTK < j1) fetch(jb + kTK);
    f32x4 s = {0.f, 0.f, 0.f, 0.f};  // keys 16 w + 4 g + r of head l15
    const bf16* ka = sk + (16 * w + l15) * ldk + 8 * g;
    const bf16* qb = sq + (16 * hg + l15) * ldk + 8 * g;
#pragma unroll 6
    for (int k = 0; k < kd; k += 32)
      s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(ka + k),
                                                  *reinterpret_cast<const bf16x8*>(qb + k), s, 0, 0, 0);
    float mx = -INFINITY;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      s[r] = jb + 16 * w + 4 * g + r < j1 ? s[r] * c2 : -INFINITY;
      mx = fmaxf(mx, s[r]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    if (g == 0) smax[w * 16 + l15] = mx;
    __syncthreads();
    float mn = m;
#pragma unroll
    for (int i = 0; i < 4; ++i) mn = fmaxf(mn, smax[i * 16 + l15]);
    const float alpha = fast_exp2(m - mn);
    m = mn;
    float sum = 0.f;
    bf16x4 pv;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float e = fast_exp2(s[r] - mn);
      sum += e;
      pv[r] = (bf16)e;
    }
    sum += __shfl_xor(sum, 16, 64);
    sum += __shfl_xor(sum, 32, 64);
    if (g == 0) ssum[w * 16 + l15] = sum;
    *reinterpret_cast<bf16x4*>(sp + l15 * (kTK + 8) + 16 * w + 4 * g) = pv;
    __syncthreads();
    l = l * alpha + (ssum[l15] + ssum[16 + l15] + ssum[32 + l15] + ssum[48 + l15]);
    float al[4];  // alpha of the accumulator's rows (heads 4 g + r)
#pragma unroll
    for (int r = 0; r < 4; ++r) al[r] = __shfl(alpha, 4 * g + r, 64);
    const bf16x8 p0 = *reinterpret_cast<const bf16x8*>(sp + l15 * (kTK + 8) + 8 * g);
    const bf16x8 p1 = *reinterpret_cast<const bf16x8*>(sp + l15 * (kTK + 8) + 32 + 8 * g);
    const int q = l15 >> 2, pp = l15 & 3;
#pragma unroll
    for (int b = 0; b < NB; ++b) {
      const int col = 16 * (w + 4 * b);
      if (col >= p.rank) break;
#pragma unroll
      for (int r = 0; r < 4; ++r) o[b][r] *= al[r];
      // 4 rows x 16 columns per lane group and read: keys 8 g + 0..3 and 8 g + 4..7 of the half
      bf16x8 v[2];
#pragma unroll
      for (int hf = 0; hf < 2; ++hf) {
        bf16* s0 = sk + (32 * hf + 8 * g + q) * ldk + col + 4 * pp;
        const bf16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) bf16x4*)s0);
        const bf16x4 hi =
            __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) bf16x4*)(s0 + 4 * ldk));
        v[hf] = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
      }
      o[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(p0, v[0], o[b], 0, 0, 0);
      o[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(p1, v[1], o[b], 0, 0, 0);
    }
  }
#pragma unroll
  for (int b = 0; b < NB; ++b) {
    const int col = 16 * (w + 4 * b) + l15;
    if (col >= p.rank) break;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int h = h0 + 4 * g + r;
      if (h < p.H) p.part_o[(((int64_t)a * p.H + h) * p.splits + split) * p.rank + col] = o[b][r];
    }
  }
  if (w == 0 && g == 0 && h0 + l15 < p.H) {
    const int64_t pi = ((int64_t)a * p.H + h0 + l15) * p.splits + split;
    p.part_ml[2 * pi] = m / kLog2e;
    p.part_ml[2 * pi + 1] = l;
  }
}

// Merges the splits of TG absorbed rows of one head and applies kUvRows rows of W_uv[h] to them (grid: heads, row groups,
// slices of W_uv[h]; every slice merges for itself).
constexpr int kUvRows = 32;

template <typename T, int TG>
__global__ __launch_bounds__(256) void latent_combine_kernel(const float* __restrict__ part_o,
                                                             const float* __restrict__ part_ml,
                                                             const T* __restrict__ uv, const int* __restrict__ atok,
                                                             T* __restrict__ out, int64_t ldo,
                                                             const T* __restrict__ gate, int64_t ldg, int n_abs, int H,
                                                             int rank, int vd, int splits) {
  extern __shared__ float so[];  // [TG][rank]
  __shared__ float sa[TG][64];
  const int h = blockIdx.x, a0 = blockIdx.y * TG;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  for (int x = w; x < TG; x += 4) {
    const int64_t pi = ((int64_t)min(a0 + x, n_abs - 1) * H + h) * splits;
    const float m = lane < splits ? part_ml[2 * (pi + lane)] : -INFINITY;
    const float l = lane < splits ? part_ml[2 * (pi + lane) + 1] : 0.f;
    const float mm = wave_max(m);
    const float e = m == -INFINITY ? 0.f : __expf(m - mm);
    const float tot = wave_sum(l * e);
    sa[x][lane] = tot > 0.f ? e / tot : 0.f;
  }
  __syncthreads();
  if (rank % 4 == 0) {
    const int rq = rank / 4;
    for (int j = threadIdx.x; j < TG * rq; j += 256) {
      const int x = j / rq, i = 4 * (j - x * rq);
      const float* po = part_o + ((int64_t)min(a0 + x, n_abs - 1) * H + h) * splits * rank + i;
      f32x4 o = {0.f, 0.f, 0.f, 0.f};
      for (int s = 0; s < splits; s += 16) {
        f32x4 v[16];
#pragma unroll
        for (int k = 0; k < 16; ++k)
          if (s + k < splits) v[k] = *reinterpret_cast<const f32x4*>(po + (int64_t)(s + k) * rank);
#pragma unroll
        for (int k = 0; k < 16; ++k)
          if (s + k < splits) o += v[k] * sa[x][s + k];
      }
      *reinterpret_cast<f32x4*>(so + x * rank + i) = o;
    }
  } else {
    for (int j = threadIdx.x; j < TG * rank; j += 256) {
      const int x = j / rank, i = j - x * rank;
      const float* po = part_o + ((int64_t)min(a0 + x, n_abs - 1) * H + h) * splits * rank + i;
      float o = 0.f;
      for (int s = 0; s < splits; ++s) o += po[(int64_t)s * rank] * sa[x][s];
      so[j] = o;
    }
  }
  __syncthreads();
  const T* u = uv + (int64_t)h * vd * rank;
  const int r0 = blockIdx.z * kUvRows + w * 8;  // a wave takes 8 value rows
  if (r0 >= vd) return;
  float acc[8][TG];
#pragma unroll
  for (int k = 0; k < 8; ++k)
#pragma unroll
    for (int x = 0; x < TG; ++x) acc[k][x] = 0.f;
  if (rank % 8 == 0) {
    for (int i = lane * 8; i < rank; i += 512) {
      float y[8][8];
#pragma unroll
      for (int k = 0; k < 8; ++k) Vec8<T>::load(u + (int64_t)min(r0 + k, vd - 1) * rank + i, y[k]);
#pragma unroll
      for (int x = 0; x < TG; ++x) {
        float z[8];
        Vec8<float>::load(so + x * rank + i, z);
#pragma unroll
        for (int k = 0; k < 8; ++k)
#pragma unroll
          for (int e = 0; e < 8; ++e) acc[k][x] += z[e] * y[k][e];
      }
    }
  } else {
    for (int i = lane; i < rank; i += 64)
#pragma unroll
      for (int k = 0; k < 8; ++k) {
        const float y = to_f(u[(int64_t)min(r0 + k, vd - 1) * rank + i]);
#pragma unroll
        for (int x = 0; x < TG; ++x) acc[k][x] += so[x * rank + i] * y;
      }
  }
#pragma unroll
  for (int x = 0; x < TG; ++x) {
    float mine = 0.f;  // lane k keeps row r0 + k
#pragma unroll
    for (int k = 0; k < 8; ++k) {
      const float v = wave_sum(acc[k][x]);
      mine = lane == k ? v : mine;
    }
    if (a0 + x < n_abs && lane < 8 && r0 + lane < vd) {
      const int64_t t = atok != nullptr ? atok[a0 + x] : a0 + x;
      if (gate != nullptr) mine *= gate_of(to_f(gate[t * ldg + h]));
      out[t * ldo + (int64_t)h * vd + r0 + lane] = from_f<T>(mine);
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------
// expanded form: flash attention over gathered keys, 32 query rows of one (sequence, head) a wave
// ---------------------------------------------------------------------------------------------------------------
struct PrefillParams {
  const bf16* q;       // [tokens, ld]: head h at column h * dk, rotated
  int64_t ldq;
  const bf16* kv;      // [rows, ldkv]: unrotated keys [H, dim], then values [H, vd]
  int64_t ldkv;
  const bf16* kr;      // [rows, ldr]: rotated key part
  int64_t ldr;
  bf16* out;           // [tokens, ldo]: head h at column h * vd
  int64_t ldo;
  const bf16* gate;    // [tokens, H] with row stride ldg (the head's output times its sigmoid), or null
  int64_t ldg;
  const int* meta;     // [n_pre][4] = {q_start, n_new, ws_row of the first key, keys before the first new token}
  int H, dim, dk, vd, window;
  float scale;
};

constexpr int BN = 64;

// DK / DV: LDS and register room; the runtime dk, vd (multiples of 16) may be smaller
// NW waves of 32 query rows; FULL: dk == DK and vd == DV
template <int DK, int DV, int NW, bool FULL>
__global__ __launch_bounds__(64 * NW) void latent_prefill_kernel(PrefillParams p) {
  constexpr int RB = 32 * NW;
  constexpr int KS = DK / 16, DT = DV / 32;
  constexpr int TK = Dim<DK>::TILE, TV = Dim<DV>::TILE;
  extern __shared__ __attribute__((aligned(1024))) char smem[];  // K[2], V[2]
  char* sK = smem;
  char* sV = smem + 2 * TK;
  const int* md = p.meta + 4 * blockIdx.z;
  const int q0 = md[0], n_new = md[1], ws0 = md[2], past = md[3];
  // the last row blocks see the most keys: they start first
  const int row_start = ((int)gridDim.x - 1 - (int)blockIdx.x) * RB;
  if (row_start >= n_new) return;
  const int head = blockIdx.y;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, h = lane >> 5;
  const int myrow = row_start + 32 * w + (lane & 31);
  const bool row_ok = myrow < n_new;
  const int tok = row_ok ? myrow : n_new - 1;
  const int qpos = past + tok;  // in key rows
  const float c = p.scale * kLog2e;
  bf16x8 qf[KS];
  {
    const bf16* qp = p.q + (int64_t)(q0 + tok) * p.ldq + (int64_t)head * p.dk + 8 * h;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      qf[ks] = bf16x8{};
      if (FULL || 16 * ks < p.dk) qf[ks] = *reinterpret_cast<const bf16x8*>(qp + 16 * ks);
    }
  }
  const int last_row = min(row_start + RB, n_new) - 1;
  const int ctx = past + last_row + 1;
  const int kt_end = (ctx + BN - 1) / BN;
  int kt_begin = 0;
  if (p.window > 0) {
    const int first = past + row_start - p.window + 1;
    kt_begin = first > 0 ? first / BN : 0;
  }
  const bf16* kbase = p.kv + (int64_t)head * p.dim;
  const bf16* vbase = p.kv + (int64_t)p.H * p.dim + (int64_t)head * p.vd;
  auto stage = [&](int kt, int buf) {
#pragma unroll
    for (int i = 0; i < 16 / NW; ++i) {
      const int n = w * (16 / NW) + i;
      const int row = 4 * n + (lane >> 4);
      const int key = min(kt * BN + row, ctx - 1);
      const int64_t kr = ws0 + key;
#pragma unroll
      for (int cc = 0; cc < Dim<DK>::NT; ++cc) {
        const int ch = 16 * cc + ((lane & 15) ^ swz(row));
        if (FULL ? 8 * ch < DK : 8 * ch < p.dk) {
          const bf16* src = 8 * ch < p.dim ? kbase + kr * p.ldkv + 8 * ch : p.kr + kr * p.ldr + (8 * ch - p.dim);
          __builtin_amdgcn_global_load_lds((gbl_void*)src, (lds_void*)(sK + buf * TK + cc * 16384 + n * 1024), 16, 0, 0);
        }
      }
#pragma unroll
      for (int cc = 0; cc < Dim<DV>::NT; ++cc) {
        const int ch = 16 * cc + ((lane & 15) ^ swz(row));
        if (FULL ? 8 * ch < DV : 8 * ch < p.vd)
          __builtin_amdgcn_global_load_lds((gbl_void*)(vbase + kr * p.ldkv + 8 * ch),
                                           (lds_void*)(sV + buf * TV + cc * 16384 + n * 1024), 16, 0, 0);
      }
    }
  };
  const int w_lo = past + min(row_start + 32 * w, n_new - 1);
  const int w_hi = past + min(row_start + 32 * w + 31, n_new - 1);
  const bool wave_active = row_start + 32 * w < n_new;
  f32x16 o[DT];
#pragma unroll
  for (int i = 0; i < DT; ++i) o[i] = f32x16{};
  float m = -INFINITY, l = 0.f;
  stage(kt_begin, 0);
  __syncthreads();
  for (int kt = kt_begin; kt < kt_end; ++kt) {
    const int buf = (kt - kt_begin) & 1;
    const char* Kt = sK + buf * TK;
    const char* Vt = sV + buf * TV;
    if (kt + 1 < kt_end) stage(kt + 1, buf ^ 1);
    const int k0 = kt * BN;
    bool skip = !wave_active || k0 > w_hi;
    if (p.window > 0 && k0 + BN - 1 <= w_lo - p.window) skip = true;
    if (!skip) {
      const bool edge = k0 + BN - 1 > w_lo || (p.window > 0 && k0 <= w_hi - p.window);
      f32x16 s[2];
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        s[t] = f32x16{};
#pragma unroll
        for (int ks = 0; ks < KS; ++ks)
          if (FULL || 16 * ks < p.dk) s[t] = mfma(rows_d(Kt, 32 * t, ks), qf[ks], s[t]);
      }
      float tmax = -INFINITY;
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          float x = s[t][r] * c;
          if (edge) {
            const int kp = k0 + 32 * t + acc_row(r, h);
            if (kp > qpos || (p.window > 0 && kp <= qpos - p.window)) x = -INFINITY;
          }
          s[t][r] = x;
          tmax = fmaxf(tmax, x);
        }
      tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
      const float mnew = fmaxf(m, tmax);
      const float muse = (mnew == -INFINITY) ? 0.f : mnew;
      const float alpha = fast_exp2(m - muse);
      float rs = 0.f;
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const float e = fast_exp2(s[t][r] - muse);
          s[t][r] = e;
          rs += e;
        }
      rs += __shfl_xor(rs, 32, 64);
      l = l * alpha + rs;
      m = mnew;
      if (__any(alpha != 1.f)) {
#pragma unroll
        for (int dt = 0; dt < DT; ++dt) o[dt] *= alpha;
      }
      const bf16x8 pb[4] = {acc_to_b<0>(s[0]), acc_to_b<1>(s[0]), acc_to_b<0>(s[1]), acc_to_b<1>(s[1])};
#pragma unroll
      for (int dt = 0; dt < DT; ++dt)
        if (FULL || 32 * dt < p.vd) {
#pragma unroll
          for (int st = 0; st < 4; ++st) o[dt] = mfma(tr_d(Vt, st, dt), pb[st], o[dt]);
        }
    }
    __syncthreads();
  }
  if (row_ok) {
    float inv = l > 0.f ? 1.f / l : 0.f;
    if (p.gate != nullptr) inv *= gate_of((float)p.gate[(int64_t)(q0 + tok) * p.ldg + head]);
    bf16* op = p.out + (int64_t)(q0 + tok) * p.ldo + (int64_t)head * p.vd;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      if (FULL || 32 * dt + 32 <= p.vd) {
        store_row_block<DV>(op, o[dt], dt, h, inv);
      } else if (32 * dt < p.vd) {  // vd = 32 k + 16: the first half of the block
#pragma unroll
        for (int g = 0; g < 2; ++g) {
          bf16x4 v4;
#pragma unroll
          for (int j = 0; j < 4; ++j) v4[j] = (bf16)(o[dt][4 * g + j] * inv);
          *reinterpret_cast<bf16x4*>(op + 32 * dt + 8 * g + 4 * h) = v4;
        }
      }
    }
  }
}

template <int DK, int DV, int NW, bool FULL>
int launch_prefill_as(const PrefillParams& p, int n_pre, int max_new, hipStream_t st) {
  constexpr int bytes = 2 * (Dim<DK>::TILE + Dim<DV>::TILE);
  static_assert(bytes <= 160 * 1024, "LDS");
  static const hipError_t attr = hipFuncSetAttribute((const void*)latent_prefill_kernel<DK, DV, NW, FULL>,
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, bytes);
  if (attr != hipSuccess) return attr;
  hipLaunchKernelGGL((latent_prefill_kernel<DK, DV, NW, FULL>), dim3((max_new + 32 * NW - 1) / (32 * NW), p.H, n_pre),
                     dim3(64 * NW), bytes, st, p);
  return hipGetLastError();
}

template <int DK, int DV>
int launch_prefill(const PrefillParams& p, int n_pre, int max_new, hipStream_t st) {
  if constexpr (DK <= 192) {  // registers for two waves per SIMD
    if (max_new > 128) {
      if (p.dk == DK && p.vd == DV) return launch_prefill_as<DK, DV, 8, true>(p, n_pre, max_new, st);
      return launch_prefill_as<DK, DV, 8, false>(p, n_pre, max_new, st);
    }
  }
  return launch_prefill_as<DK, DV, 4, false>(p, n_pre, max_new, st);
}

size_t decode_lds(int rank, int rot, int hg) {
  const int kd = (rank + rot + 31) & ~31;
  return (size_t)(kTK + 16 * hg) * (kd + 8) * 2 + hg * (16 * (kTK + 8) * 2 + 128 * 4);
}

template <int HG, int NCH, int NB>
int launch_decode(const DecodeParams<bf16>& p, int n_abs, hipStream_t st) {
  const size_t lds = decode_lds(p.rank, p.rot, HG);
  static const hipError_t attr = hipFuncSetAttribute((const void*)latent_decode_mfma_kernel<HG, NCH, NB>,
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
  if (attr != hipSuccess) return attr;
  hipLaunchKernelGGL((latent_decode_mfma_kernel<HG, NCH, NB>),
                     dim3(p.splits, (p.H + 16 * HG - 1) / (16 * HG), n_abs), dim3(256 * HG), lds, st, p);
  return hipGetLastError();
}

// heads of one workgroup / 16
int decode_hg(int H, int rank, int rot) {
  const int kd = (rank + rot + 31) & ~31;
  return H > 16 && kd <= 640 && rank <= 512 ? 2 : 1;
}

}  // namespace

HDS_EXPORT int hds_latent_prep(int dtype, void* q, int64_t ldq, const void* c, int64_t ldc, const float* norm,
                               const float* cos_t, const float* sin_t, void* cache, const int* tok_seq, const int* tok_pos,
                               const int* tables, const int* ws_row, void* ws, const void* uk, const int* atok,
                               void* qa, int n_tok, int n_abs, int n_pos, int max_blocks, int block_size, int H,
                               int dim, int rot, int rdims, int rank, float eps, hipStream_t st) {
  if (n_tok <= 0) return 0;
  if (H < 1 || dim < 0 || rot < 0 || rdims < 0 || rdims > rot || rdims % 2 || rank < 1 || n_pos < 1 || n_abs < 0 ||
      n_abs > n_tok || block_size < 1 || ldq < (int64_t)H * (dim + rot) || ldc < rank + rot || (n_abs > 0 && (!qa || !uk)))
    return hipErrorInvalidValue;
  const bool v8 = dim % 8 == 0 && rot % 8 == 0 && rdims % 8 == 0 && rank % 8 == 0 && rank <= 2048 && ldq % 8 == 0 && ldc % 8 == 0 &&
                  (uintptr_t)q % 16 == 0 && (uintptr_t)c % 16 == 0 && (uintptr_t)cos_t % 16 == 0 && (uintptr_t)sin_t % 16 == 0;
  const int64_t cblocks = v8 ? (rank + kAbsCols - 1) / kAbsCols : 1;
  const int tg = v8 && n_abs == 1 ? 1 : kAbsTok;
  const int64_t grid = n_tok + (int64_t)((n_abs + tg - 1) / tg) * H * cblocks;
  const size_t lds = sizeof(float) * (kAbsTok * dim + 16 + (v8 ? 4 * kAbsTok * kAbsCols : 0));
  if (grid > 0x7fffffff || lds > 64 * 1024) return hipErrorInvalidValue;
#define HDS_LP(TT)                                                                                                   \
  {                                                                                                                  \
    PrepParams<TT> p{(TT*)q, ldq, (const TT*)c, ldc, norm, cos_t, sin_t, (TT*)cache, tok_seq, tok_pos, tables,       \
                     ws_row, (TT*)ws, (const TT*)uk, atok, (TT*)qa, n_tok, n_abs, n_pos, max_blocks, block_size, H, dim, rot, rdims, \
                     rank, eps};                                                                                     \
    if (v8 && n_abs == 0)                                                                                            \
      hipLaunchKernelGGL((latent_prep8_kernel<TT, 0>), dim3((unsigned)grid), dim3(256), 64, st, p);                  \
    else if (v8 && n_abs == 1)                                                                                       \
      hipLaunchKernelGGL((latent_prep8_kernel<TT, 1>), dim3((unsigned)grid), dim3(256), lds, st, p);                 \
    else if (v8)                                                                                                     \
      hipLaunchKernelGGL((latent_prep8_kernel<TT, kAbsTok>), dim3((unsigned)grid), dim3(256), lds, st, p);           \
    else                                                                                                             \
      hipLaunchKernelGGL(latent_prep_kernel<TT>, dim3((unsigned)grid), dim3(256), lds, st, p);                       \
  }
  if (dtype == kBF16) HDS_LP(bf16) else if (dtype == kF32) HDS_LP(float) else return hipErrorInvalidValue;
#undef HDS_LP
  return hipGetLastError();
}

HDS_EXPORT int hds_latent_decode_mfma_ok(int rank, int rot) {
  return rank % 8 == 0 && rot % 8 == 0 && rank >= 8 && rank + rot <= 960;
}

// key splits of one absorbed row: about one workgroup per CU, >= 128 keys each (the partial sums of a split are as
// large as 128 cached rows of a wide latent), <= 64 (one wave merges them)
HDS_EXPORT int hds_latent_decode_splits(int n_abs, int H, int rank, int rot, int mfma, int max_keys) {
  const int per = mfma ? 16 * decode_hg(H, rank, rot) : 1;
  const int64_t groups = (int64_t)n_abs * ((H + per - 1) / per);
  int64_t s = (256 + groups - 1) / groups;
  const int by_len = (max_keys + 127) / 128;
  s = s < by_len ? s : by_len;
  return s < 1 ? 1 : (s > 64 ? 64 : (int)s);
}

HDS_EXPORT int hds_latent_decode(int dtype, const void* qa, const void* cache, float* part_o, float* part_ml,
                                 const int* atok, const int* tok_seq, const int* tok_pos, const int* tables,
                                 int max_blocks, int block_size, int n_abs, int H, int rank, int rot, int splits,
                                 int window, float scale, int mfma, hipStream_t st) {
  if (n_abs <= 0) return 0;
  if (splits < 1 || splits > 64 || H < 1 || rank < 1 || rot < 0 || block_size < 1 || window < 0 || n_abs > 65535 ||
      H > 65535)
    return hipErrorInvalidValue;
  if (mfma) {
    if (dtype != kBF16 || !hds_latent_decode_mfma_ok(rank, rot)) return hipErrorInvalidValue;
    DecodeParams<bf16> p{(const bf16*)qa, (const bf16*)cache, part_o, part_ml, atok, tok_seq, tok_pos, tables,
                         max_blocks, block_size, H, rank, rot, splits, window, scale};
    const int kd = (rank + rot + 31) & ~31;
    const bool two = decode_hg(H, rank, rot) == 2;
    if (kd <= 128) return two ? launch_decode<2, 2, 2>(p, n_abs, st) : launch_decode<1, 4, 2>(p, n_abs, st);
    if (kd <= 320 && rank <= 256) return two ? launch_decode<2, 5, 4>(p, n_abs, st) : launch_decode<1, 10, 4>(p, n_abs, st);
    if (kd <= 640 && rank <= 512) return two ? launch_decode<2, 10, 8>(p, n_abs, st) : launch_decode<1, 20, 8>(p, n_abs, st);
    return launch_decode<1, 30, 15>(p, n_abs, st);
  }
  const size_t lds = sizeof(float) * (size_t)(2 * rank + rot + kGenKeys);
  if (lds > 64 * 1024) return hipErrorInvalidValue;
#define HDS_LD(TT)                                                                                              \
  {                                                                                                             \
    DecodeParams<TT> p{(const TT*)qa, (const TT*)cache, part_o, part_ml, atok, tok_seq, tok_pos, tables,       \
                       max_blocks, block_size, H, rank, rot, splits, window, scale};                            \
    hipLaunchKernelGGL(latent_decode_plain_kernel<TT>, dim3(splits, H, n_abs), dim3(256), lds, st, p);          \
  }
  if (dtype == kBF16) HDS_LD(bf16) else if (dtype == kF32) HDS_LD(float) else return hipErrorInvalidValue;
#undef HDS_LD
  return hipGetLastError();
}

HDS_EXPORT int hds_latent_combine(int dtype, const float* part_o, const float* part_ml, const void* uv,
                                  const int* atok, void* out, int64_t ldo, const void* gate, int64_t ldg, int n_abs,
                                  int H, int rank, int vd, int splits, hipStream_t st) {
  if (n_abs <= 0) return 0;
  if (splits < 1 || splits > 64 || vd < 1 || n_abs > 65535 || rank > 8192) return hipErrorInvalidValue;
#define HDS_LC(TT, TG)                                                                                               \
  hipLaunchKernelGGL((latent_combine_kernel<TT, TG>), dim3(H, (n_abs + TG - 1) / TG, (vd + kUvRows - 1) / kUvRows), \
                     dim3(256), TG * rank * sizeof(float), st, part_o, part_ml, (const TT*)uv, atok, (TT*)out, ldo, \
                     (const TT*)gate, ldg, n_abs, H, rank, vd, splits)
  const bool four = n_abs >= 4 && rank <= 2048;
  if (dtype == kBF16) {
    if (four) HDS_LC(bf16, 4); else HDS_LC(bf16, 1);
  } else if (dtype == kF32) {
    if (four) HDS_LC(float, 4); else HDS_LC(float, 1);
  } else {
    return hipErrorInvalidValue;
  }
#undef HDS_LC
  return hipGetLastError();
}

// bf16; dk = dim + rot and vd multiples of 16, dim, rot and rank multiples of 8 (16-B rows of every operand)
HDS_EXPORT int hds_latent_prefill_ok(int dim, int rot, int rank, int vd) {
  const int dk = dim + rot;
  return dk % 16 == 0 && vd % 16 == 0 && dim % 8 == 0 && rot % 8 == 0 && rank % 8 == 0 && dk >= 16 && vd >= 16 &&
         dk <= 256 && vd <= 256;
}

HDS_EXPORT int hds_latent_prefill(const void* q, int64_t ldq, const void* kv, int64_t ldkv, const void* kr,
                                  int64_t ldr, void* out, int64_t ldo, const void* gate, int64_t ldg, const int* meta,
                                  int n_pre, int max_new, int H, int dim, int rot, int rank, int vd, int window,
                                  float scale, hipStream_t st) {
  if (n_pre <= 0 || max_new <= 0) return 0;
  if (!hds_latent_prefill_ok(dim, rot, rank, vd) || ldq % 8 || ldkv % 8 || ldr % 8 || ldo % 8 || H > 65535 ||
      n_pre > 65535 || window < 0)
    return hipErrorInvalidValue;
  PrefillParams p{(const bf16*)q, ldq, (const bf16*)kv, ldkv, (const bf16*)kr, ldr, (bf16*)out, ldo, (const bf16*)gate, ldg, meta, H, dim,
                  dim + rot, vd, window, scale};
  const int dk = dim + rot;
  if (dk <= 64 && vd <= 64) return launch_prefill<64, 64>(p, n_pre, max_new, st);
  if (dk <= 128 && vd <= 128) return launch_prefill<128, 128>(p, n_pre, max_new, st);
  if (dk <= 192 && vd <= 128) return launch_prefill<192, 128>(p, n_pre, max_new, st);
  return launch_prefill<256, 256>(p, n_pre, max_new, st);
}
