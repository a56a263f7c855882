// Serving kernels over the paged (blocked) KV cache: fused RoPE + KV scatter, and ragged
// prefill/decode attention that reads K/V through per-sequence block tables.
//
// Capability parity: deepspeed/inference/v2/kernels/ragged_ops/linear_blocked_kv_rotary
// (`kv_rotary_pos_kernel`, SURVEY §2.11 K31 -- also the only kernel the HCache `restore_kv`
// path runs) and blocked_flash (`run_mha_fwd` over AttentionAtoms, K32, a prebuilt NVIDIA-only
// library in the reference).
//
// Cache layout per layer (same as the reference BlockedKVCache): [num_blocks, block_size, 2, Hkv, D]
// (K then V for each slot). Key and value heads may differ in size: a slot is then [Hkv * DK | Hkv * DV], the same
// layout when DK == DV. Any block_size works: every staged tile row computes its own
// (block, slot) address, and LDS-DMA takes a per-lane global source address.
//
// Head dims: every multiple of 16 up to 256 that flash_attn.hip instantiates (HDS_PAGED_DIMS below), via the
// generic tile helpers of attn_common.h; other sizes that are multiples of 8 run the same kernel on zero-padded tiles,
// float32 and everything else a plain kernel. The RoPE scatter takes any head_dim % 4 == 0 with a rotary prefix
// of rot_dim (% 8 == 0) dims -- partial rotary (Phi, GPT-NeoX) rotates the prefix and copies the rest.
//
// Attention work unit ("atom"): (sequence, kv head, 128 packed rows). Rows pack the G = Hq/Hkv
// query heads that share a kv head with the tokens of the chunk (row = token * G + head_in_group),
// so K/V of a kv head are read ONCE for all of its query heads -- for decode (1 token) one wave
// serves the whole GQA group from a single pass over the sequence's KV blocks.
//
// Options of all attention kernels: a sliding window, in front of which the sequence's first `keep` positions stay visible; chunks, runs of positions counted from the sequence's start that see
// only themselves; a soft cap of the scores, cap * tanh(score / cap); a sink, one score per query head that joins the
// softmax denominator but has no key and no value; an output gate, one value per token and query head (or per element of
// the head's output) whose sigmoid multiplies it. head_norm_scatter is the counterpart of the RoPE scatter for heads that
// are not rotated: optional RMS norms of q and k, optional mixing of the values with another layer's.
#include "attn_common.h"

using namespace hds;
using namespace hds::attn;

namespace {

constexpr int BN = 64;
constexpr float kLog2e = 1.4426950408889634f;

// ------------------------------------------------------------------------------------------
// fused RoPE (q in place, k rotated into the cache) + V copy into the cache
// ------------------------------------------------------------------------------------------
template <typename T>
struct Vec4 {  // 4 x 16-bit elements = one 8-byte access
  typedef uint32_t u2 __attribute__((ext_vector_type(2)));
  __device__ __forceinline__ static void load(const T* p, float (&v)[4]) {
    const u2 r = *reinterpret_cast<const u2*>(p);
    const T* e = reinterpret_cast<const T*>(&r);
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = (float)e[i];
  }
  __device__ __forceinline__ static void store(T* p, const float (&v)[4]) {
    u2 r;
    T* e = reinterpret_cast<T*>(&r);
#pragma unroll
    for (int i = 0; i < 4; ++i) e[i] = (T)v[i];
    *reinterpret_cast<u2*>(p) = r;
  }
};

// per head: rot/8 rotation groups of 4 pairs (i, i + rot/2), then (D - rot)/4 plain 4-element chunks. 4-element
// granularity covers every rotary prefix the HF families use (Phi partial_rotary 0.4 / 0.5 of 80 -> 32 / 40).
template <typename T>
__global__ __launch_bounds__(256) void kv_rope_scatter_kernel(T* __restrict__ qkv, int64_t sq, T* __restrict__ cache,
                                                              const int* __restrict__ tok_seq,
                                                              const int* __restrict__ tok_pos,
                                                              const int* __restrict__ block_tables, int max_blocks,
                                                              const float* __restrict__ cos_t,
                                                              const float* __restrict__ sin_t, int n_tok, int hq,
                                                              int hkv, int D, int rot, int block_size, int rotate_q,
                                                              int do_rope) {
  const int half = rot / 2;
  const int nrot = rot / 8;
  const int gph = nrot + (D - rot) / 4;
  const int heads = hq + 2 * hkv;
  const int64_t total = (int64_t)n_tok * heads * gph;
  for (int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x; idx < total; idx += (int64_t)gridDim.x * 256) {
    const int t = (int)(idx / (heads * gph));
    const int rem = (int)(idx - (int64_t)t * heads * gph);
    const int h = rem / gph, g = rem - h * gph;
    if (h < hq && !rotate_q) continue;
    const int pos = tok_pos[t];
    T* src = qkv + (int64_t)t * sq + (int64_t)h * D;
    T* dst = nullptr;
    if (h >= hq) {
      const int kv = (h < hq + hkv) ? 0 : 1;
      const int hk = h - hq - kv * hkv;
      const int seq = tok_seq[t];
      const int blk = block_tables[(int64_t)seq * max_blocks + pos / block_size];
      const int slot = pos % block_size;
      dst = cache + ((((int64_t)blk * block_size + slot) * 2 + kv) * hkv + hk) * D;
    }
    if (g >= nrot) {  // un-rotated tail (and every V chunk past the rotary prefix)
      if (dst == nullptr) continue;
      const int c0 = rot + (g - nrot) * 4;
      float a[4];
      Vec4<T>::load(src + c0, a);
      Vec4<T>::store(dst + c0, a);
      continue;
    }
    float a[4], b[4];
    Vec4<T>::load(src + g * 4, a);
    Vec4<T>::load(src + half + g * 4, b);
    if (h < hq + hkv && do_rope) {
      const f32x4 c = *reinterpret_cast<const f32x4*>(cos_t + (int64_t)pos * half + g * 4);
      const f32x4 sn = *reinterpret_cast<const f32x4*>(sin_t + (int64_t)pos * half + g * 4);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float oa = a[j] * c[j] - b[j] * sn[j];
        const float ob = b[j] * c[j] + a[j] * sn[j];
        a[j] = oa;
        b[j] = ob;
      }
    }
    T* out = dst != nullptr ? dst : src;  // q rotates in place
    Vec4<T>::store(out + g * 4, a);
    Vec4<T>::store(out + half + g * 4, b);
  }
}

// ------------------------------------------------------------------------------------------
// per-head RMS norm of q (in place) and k (into the cache) + V copy into the cache
// ------------------------------------------------------------------------------------------
template <typename T>
struct HeadNormParams {
  T* qkv;  // [tokens, ld]: hq query heads of dk, hkv key heads of dk, hkv value heads of dv
  int64_t ld;
  const float* qn;  // [dk] or null: q stays as it is
  const float* kn;
  T* cache;
  const int* tok_seq;
  const int* tok_pos;
  const int* tables;
  int n_tok, max_blocks, block_size, hq, hkv, dk, dv;
  float eps;
  const T* v0;  // [tokens, ldv0] values of another layer, or null: v <- v + mix * (v0 - v)
  int64_t ldv0;
  const float* mix;
};

template <typename T>
__device__ __forceinline__ T* cache_slot(const HeadNormParams<T>& p, int t) {
  const int pos = p.tok_pos[t];
  const int blk = p.tables[(int64_t)p.tok_seq[t] * p.max_blocks + pos / p.block_size];
  return p.cache + ((int64_t)blk * p.block_size + pos % p.block_size) * p.hkv * (p.dk + p.dv);
}

// LPH lanes per head, 8 elements each (dk, dv and ld multiples of 8)
template <typename T, int LPH>
__global__ __launch_bounds__(256) void head_norm_scatter8_kernel(HeadNormParams<T> p) {
  constexpr int HPB = 256 / LPH;
  const int heads = p.hq + 2 * p.hkv;
  const int64_t item = (int64_t)blockIdx.x * HPB + threadIdx.x / LPH;
  const int c = 8 * (threadIdx.x % LPH);
  const bool live = item < (int64_t)p.n_tok * heads;  // no early exit: the lanes of a head reduce together
  const int t = live ? (int)(item / heads) : 0, h = live ? (int)(item - (int64_t)t * heads) : 0;
  const bool is_v = h >= p.hq + p.hkv;
  const int d = is_v ? p.dv : p.dk;
  const int off = is_v ? (p.hq + p.hkv) * p.dk + (h - p.hq - p.hkv) * p.dv : h * p.dk;
  const bool ok = live && c < d;
  T* src = p.qkv + (int64_t)t * p.ld + off + c;
  float v[8];
  float ss = 0.f;
  if (ok) {
    Vec8<T>::load(src, v);
#pragma unroll
    for (int i = 0; i < 8; ++i) ss += v[i] * v[i];
  }
#pragma unroll
  for (int o = LPH / 2; o >= 1; o >>= 1) ss += __shfl_xor(ss, o, 64);
  if (!ok) return;
  const float* w = is_v ? nullptr : (h < p.hq ? p.qn : p.kn);
  if (w != nullptr) {
    const float rs = 1.f / sqrtf(ss / (float)p.dk + p.eps);
    float n[8];
    Vec8<float>::load(w + c, n);
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] *= rs * n[i];
  }
  if (is_v && p.v0 != nullptr) {
    const float lam = *p.mix;
    float o[8];
    Vec8<T>::load(p.v0 + (int64_t)t * p.ldv0 + (h - p.hq - p.hkv) * p.dv + c, o);
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = (1.f - lam) * v[i] + lam * o[i];
  }
  if (h < p.hq) {
    if (w != nullptr) Vec8<T>::store(src, v);
  } else {
    Vec8<T>::store(cache_slot(p, t) + off - p.hq * p.dk + c, v);
  }
}

// any sizes: one wave per head
template <typename T>
__global__ __launch_bounds__(256) void head_norm_scatter_kernel(HeadNormParams<T> p) {
  const int heads = p.hq + 2 * p.hkv;
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= (int64_t)p.n_tok * heads) return;
  const int lane = threadIdx.x & 63, t = (int)(item / heads), h = (int)(item - (int64_t)t * heads);
  const bool is_v = h >= p.hq + p.hkv;
  const int d = is_v ? p.dv : p.dk;
  const int off = is_v ? (p.hq + p.hkv) * p.dk + (h - p.hq - p.hkv) * p.dv : h * p.dk;
  T* src = p.qkv + (int64_t)t * p.ld + off;
  const float* w = is_v ? nullptr : (h < p.hq ? p.qn : p.kn);
  T* dst = h < p.hq ? src : cache_slot(p, t) + off - p.hq * p.dk;
  float rs = 1.f;
  if (w != nullptr) {
    float ss = 0.f;
    for (int i = lane; i < d; i += 64) ss += to_f(src[i]) * to_f(src[i]);
    rs = 1.f / sqrtf(wave_sum(ss) / (float)d + p.eps);
  }
  if (is_v && p.v0 != nullptr) {
    const float lam = *p.mix;
    const T* o = p.v0 + (int64_t)t * p.ldv0 + (h - p.hq - p.hkv) * p.dv;
    for (int i = lane; i < d; i += 64) dst[i] = from_f<T>((1.f - lam) * to_f(src[i]) + lam * to_f(o[i]));
    return;
  }
  for (int i = lane; i < d; i += 64) dst[i] = from_f<T>(w != nullptr ? to_f(src[i]) * rs * w[i] : to_f(src[i]));
}

// ------------------------------------------------------------------------------------------
// paged attention (ragged prefill + decode)
// ------------------------------------------------------------------------------------------
// A sequence's slots: position -> (block, slot) without an integer division per access. The reciprocal is exact for
// positions below 2^32 / block_size (longer tables divide).
struct PageTable {
  const int* table;
  int size;
  uint32_t inv;  // 0: divide
  __device__ __forceinline__ PageTable(const int* t, int block_size, int max_blocks) : table(t), size(block_size) {
    inv = 0xFFFFFFFFu / (uint32_t)block_size + 1u;  // 0 for blocks of one slot
    if ((uint64_t)max_blocks * block_size * block_size >> 32) inv = 0;
  }
  __device__ __forceinline__ int block(int pos) const {
    return inv != 0 ? (int)__umulhi((uint32_t)pos, inv) : pos / size;
  }
  __device__ __forceinline__ int64_t slot(int pos) const {
    const int b = block(pos);
    return (int64_t)table[b] * size + (pos - b * size);
  }
};

__device__ __forceinline__ float gate_of(float g) { return 1.f / (1.f + __expf(-g)); }

// cap * tanh(x / cap)
__device__ __forceinline__ float soft_cap(float x, float cap) { return cap * tanhf(x / cap); }
// the same in the log2 domain of the matrix-core kernel: cap2 = cap * log2(e), inv2 = 2 / cap, x and the result scaled by
// log2(e); tanh(y) = 1 - 2 / (exp(2 y) + 1)
__device__ __forceinline__ float soft_cap2(float x, float cap2, float inv2) {
  return cap2 - 2.f * cap2 * __builtin_amdgcn_rcpf(fast_exp2(x * inv2) + 1.f);
}

// the first position that position pos sees (window, chunk: 0 for none), apart from the kept ones below `keep`
__device__ __forceinline__ int first_key(int pos, int window, int chunk) {
  int lo = window > 0 ? max(0, pos + 1 - window) : 0;
  if (chunk > 0) lo = max(lo, pos - pos % chunk);
  return lo;
}

struct PagedParams {
  const bf16* q;  // [T, Hq, DK] rows with token stride sq
  int64_t sq;
  const bf16* cache;  // layer base: [num_blocks, block_size, Hkv * DK | Hkv * DV]
  bf16* o;            // [T, Hq, DV] rows with token stride so
  int64_t so;
  const int* atoms;   // [n_atoms][3] = {seq, kv_head, row_start}
  const int* seq_meta;  // [n_seqs][3] = {q_start, n_new, seen}
  const int* block_tables;
  int max_blocks;
  int block_size;
  int hq, hkv;
  int dk, dv;  // read by the padded kernels only
  float scale;
  int window, chunk, keep;
  float softcap;      // 0: none
  const float* sink;  // [Hq] or null
  const bf16* gate;   // [T, Hq * gw] with token stride sg, or null
  int64_t sg;
  int gw;             // 1: a gate per head, dv: one per element
};

// DK / DV: head sizes, or with PAD their upper bounds (tiles zero-padded to them; the sizes are multiples of 8)
// Two workgroups per CU where their LDS fits
template <int DK, int DV>
constexpr int atom_waves() { return Dim<DK>::TILE + Dim<DV>::TILE <= 32768 ? 2 : 1; }

template <int DK, int DV, int NW, bool PAD>
__global__ __launch_bounds__(64 * NW, (atom_waves<DK, DV>())) void paged_attn_kernel(PagedParams p) {
  constexpr int KS = Dim<DK>::KS, DT = Dim<DV>::DT, TLK = Dim<DK>::TILE, TLV = Dim<DV>::TILE;
  __shared__ __attribute__((aligned(16))) char smem[2 * TLK + 2 * TLV];  // K[2], V[2]
  const int dk = PAD ? p.dk : DK, dv = PAD ? p.dv : DV;
  const int* at = p.atoms + blockIdx.x * 3;
  const int seq = at[0], hk = at[1], row_start = at[2];
  const int q_start = p.seq_meta[seq * 3], n_new = p.seq_meta[seq * 3 + 1], seen = p.seq_meta[seq * 3 + 2];
  const int G = p.hq / p.hkv;
  const int n_rows = n_new * G;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, h = lane >> 5;
  const int myrow = row_start + 32 * w + (lane & 31);
  const bool row_ok = myrow < n_rows;
  const int rr = row_ok ? myrow : n_rows - 1;
  const int tok = rr / G, head = hk * G + rr % G;
  const int qpos = seen + tok;  // absolute position of this row's query
  const float c = p.scale * kLog2e;
  const bool bounded = p.window > 0 || p.chunk > 0;
  const int lo = first_key(qpos, p.window, p.chunk);
  const int* table = p.block_tables + (int64_t)seq * p.max_blocks;
  const int64_t kv_row = (int64_t)p.hkv * (dk + dv);  // elements between consecutive slots

  if constexpr (PAD) {  // staging fills the chunks below dk / dv only: the rest stays zero
    for (int i = threadIdx.x; i < (2 * TLK + 2 * TLV) / 16; i += 64 * NW) reinterpret_cast<u32x4*>(smem)[i] = u32x4{};
    __syncthreads();
  }
  bf16x8 qf[KS];
  {
    const bf16* qp = p.q + (int64_t)(q_start + tok) * p.sq + (int64_t)head * dk + 8 * h;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      if constexpr (PAD) {
        qf[ks] = bf16x8{};
        if (16 * ks + 8 * h < dk) qf[ks] = *reinterpret_cast<const bf16x8*>(qp + 16 * ks);
      } else {
        qf[ks] = *reinterpret_cast<const bf16x8*>(qp + 16 * ks);
      }
    }
  }
  // last query position covered by this workgroup (rows are token-major)
  const int last_row = min(row_start + 32 * NW, n_rows) - 1;
  const int wg_qpos_max = seen + last_row / G;
  const int ctx = wg_qpos_max + 1;
  const int kt_end = (ctx + BN - 1) / BN;
  const int kt_begin = bounded ? first_key(seen + row_start / G, p.window, p.chunk) / BN : 0;
  const int kept = bounded ? min((p.keep + BN - 1) / BN, kt_begin) : 0;  // tiles of kept keys ahead of the others
  const int n_tiles = kt_end - kt_begin + kept;
  auto tile_at = [&](int i) { return i < kept ? i : i - kept + kt_begin; };
  auto rowp = [&](int kt, int off) {
    return [=](int row) {
      int pos = kt * BN + row;
      pos = pos < ctx ? pos : ctx - 1;
      const int blk = table[pos / p.block_size];
      return p.cache + ((int64_t)blk * p.block_size + pos % p.block_size) * kv_row + off;
    };
  };
  const int koff = hk * dk, voff = p.hkv * dk + hk * dv;
  auto stage = [&](int buf, int kt) {
    if constexpr (PAD) {
      stage_tile_n<NW, DK>(smem + buf * TLK, rowp(kt, koff), dk / 8);
      stage_tile_n<NW, DV>(smem + 2 * TLK + buf * TLV, rowp(kt, voff), dv / 8);
    } else {
      stage_tile_d<NW, DK>(smem + buf * TLK, rowp(kt, koff));
      stage_tile_d<NW, DV>(smem + 2 * TLK + buf * TLV, rowp(kt, voff));
    }
  };
  const int w_row_lo = row_start + 32 * w;
  const int w_qpos_lo = seen + min(w_row_lo, n_rows - 1) / G;
  const int w_qpos_hi = seen + min(w_row_lo + 31, n_rows - 1) / G;
  const bool wave_active = w_row_lo < n_rows;
  const int w_lo = bounded ? first_key(w_qpos_lo, p.window, p.chunk) : 0;

  f32x16 o[DT];
#pragma unroll
  for (int i = 0; i < DT; ++i) o[i] = f32x16{};
  // the sink is a key of its own score and no value, seen before all others
  float m = -INFINITY, l = 0.f;
  if (p.sink != nullptr) {
    m = p.sink[head] * kLog2e;
    l = 1.f;
  }

  stage(0, tile_at(0));
  __syncthreads();
  for (int it = 0; it < n_tiles; ++it) {
    const int buf = it & 1, kt = tile_at(it);
    const char* Kt = smem + buf * TLK;
    const char* Vt = smem + 2 * TLK + buf * TLV;
    if (it + 1 < n_tiles) stage(buf ^ 1, tile_at(it + 1));
    const int k0 = kt * BN;
    bool skip = !wave_active || k0 > w_qpos_hi;
    if (k0 + BN - 1 < w_lo && k0 >= p.keep) skip = true;
    if (!skip) {
      f32x16 s[2];
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        s[t] = f32x16{};
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) s[t] = mfma(rows_d(Kt, 32 * t, ks), qf[ks], s[t]);
      }
      if (p.softcap > 0.f) {  // (s * c holds the score times log2(e))
        const float cap2 = p.softcap * kLog2e / c, inv2 = 2.f * c / p.softcap;
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
          for (int r = 0; r < 16; ++r) s[t][r] = soft_cap2(s[t][r], cap2, inv2);
      }
      float tmax = -INFINITY;
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int kp = k0 + 32 * t + acc_row(r, h);
          float x = s[t][r] * c;
          if (kp > qpos || !row_ok || (kp < lo && kp >= p.keep)) x = -INFINITY;
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
#pragma unroll
        for (int st = 0; st < 4; ++st) o[dt] = mfma(tr_d(Vt, st, dt), pb[st], o[dt]);
    }
    __syncthreads();
  }
  if (row_ok) {
    float inv = l > 0.f ? 1.f / l : 0.f;
    const bf16* gp = p.gate == nullptr ? nullptr : p.gate + (int64_t)(q_start + tok) * p.sg + (int64_t)head * p.gw;
    if (gp != nullptr && p.gw == 1) {
      inv *= gate_of((float)*gp);
    } else if (gp != nullptr) {  // registers 4 g .. 4 g + 3 of a block are neighbouring columns
#pragma unroll
      for (int dt = 0; dt < DT; ++dt)
#pragma unroll
        for (int g = 0; g < 4; ++g) {
          const int col = 32 * dt + 8 * g + 4 * h;
          if (col < dv) {
            const bf16x4 gv = *reinterpret_cast<const bf16x4*>(gp + col);
#pragma unroll
            for (int j = 0; j < 4; ++j) o[dt][4 * g + j] *= gate_of((float)gv[j]);
          }
        }
    }
    bf16* op = p.o + (int64_t)(q_start + tok) * p.so + (int64_t)head * dv;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      if constexpr (PAD) store_row_block_n(op, o[dt], dt, h, inv, dv);
      else store_row_block<DV>(op, o[dt], dt, h, inv);
    }
  }
}

// ------------------------------------------------------------------------------------------
// single tokens: split-K ("flash decoding") over the paged cache
// ------------------------------------------------------------------------------------------
// The atom kernel above would run one 4-wave workgroup per (sequence, kv head) for a lone new token --
// 8 workgroups for a single Llama-3-8B sequence, each walking the whole context on a mostly empty 128-row MFMA tile
// (35 us per layer at 540 keys, profiles/r3). Decode is a K/V stream, so this kernel is built like decode_attn.hip:
// grid (splits, Hkv x blocks of GM query heads, tokens), a workgroup serves its query heads from ONE read of its key
// range, 16-B loads with LPK lanes per key (8 elements of a key and of a value each), U keys per lane group in
// flight while as many are used (the stream is bound by the bytes in flight), online softmax in registers, lane groups and waves merged by max / rescale, splits merged
// by a combine kernel through fp32 partials. The key range comes from device-side metadata (and covers only the
// window), so one launch shape serves every step of a HIP-graph decode.
constexpr int kDecGMax = 8;

template <typename T>
struct PagedDecodeParams {
  const T* q;  // [T, Hq, DK] rows with token stride sq
  int64_t sq;
  const T* cache;  // [num_blocks, block_size, Hkv * DK | Hkv * DV]
  T* o;            // [T, Hq, DV] rows with token stride so
  int64_t so;
  float* part_o;   // [n, Hq, splits, DV]
  float* part_ml;  // [n, Hq, splits, 2]
  // the n tokens: seq_meta [n][3] = {q_start, n_new (1), seen}, one sequence each; or, with seq_meta null, rows
  // toks[i] (null: i) of the step's tok_seq / tok_pos
  const int* seq_meta;
  const int* toks;
  const int* tok_seq;
  const int* tok_pos;
  const int* block_tables;
  int max_blocks, block_size, hq, hkv, dk, dv, splits;
  float scale;
  int window, chunk, keep;
  float softcap;      // 0: none
  const float* sink;  // [Hq] or null
  const T* gate;      // [T, Hq * gw] with token stride sg, or null
  int64_t sg;
  int gw;             // 1: a gate per head, dv: one per element
  // splits > 1: one int per (token, kv head), zero between launches. Non-null: the last workgroup of a
  // (token, kv head) to finish merges the splits itself (no combine launch) and resets its counter to 0, so a
  // HIP-graph replay finds it zeroed again.
  int* counters;
};

struct DecodeToken {
  int row, seq, pos;
};

template <typename T>
__device__ __forceinline__ DecodeToken decode_token(const PagedDecodeParams<T>& p, int b) {
  if (p.seq_meta != nullptr) return {p.seq_meta[3 * b], b, p.seq_meta[3 * b + 2]};
  const int t = p.toks != nullptr ? p.toks[b] : b;
  return {t, p.tok_seq[t], p.tok_pos[t]};
}

// this split's keys: an equal share of what the token sees, counted without the gap between the kept keys and the others
struct DecodeKeys {
  int j0, j1, keep, gap;
  __device__ __forceinline__ int pos(int j) const { return j < keep ? j : j + gap; }
};
template <typename T>
__device__ __forceinline__ DecodeKeys decode_keys(const PagedDecodeParams<T>& p, int pos, int split) {
  const int gap = max(first_key(pos, p.window, p.chunk) - p.keep, 0), n = pos + 1 - gap;
  const int per = (n + p.splits - 1) / p.splits;
  return {split * per, min(n, split * per + per), p.keep, gap};
}

// factor of head h's weighted value sum whose softmax so far has maximum m and denominator l
template <typename T>
__device__ __forceinline__ float decode_factor(const PagedDecodeParams<T>& p, int row, int h, float m, float l) {
  float f = 1.f;
  if (p.sink != nullptr) {
    const float mm = fmaxf(m, p.sink[h]);
    f = m == -INFINITY ? 0.f : __expf(m - mm);
    l = l * f + __expf(p.sink[h] - mm);
  }
  f = l > 0.f ? f / l : 0.f;
  return p.gate != nullptr && p.gw == 1 ? f * gate_of(to_f(p.gate[(int64_t)row * p.sg + h])) : f;
}

// gate of element d of head h's output, where every element has its own (else 1; the head's gate is in decode_factor)
template <typename T>
__device__ __forceinline__ float decode_gate(const PagedDecodeParams<T>& p, int row, int h, int d) {
  return p.gate != nullptr && p.gw > 1 ? gate_of(to_f(p.gate[(int64_t)row * p.sg + (int64_t)h * p.gw + d])) : 1.f;
}

template <typename T>
__device__ __forceinline__ void decode_merge_splits(const PagedDecodeParams<T>& p, int b, int h, int d, int row) {
  const float* pm = p.part_ml + ((int64_t)b * p.hq + h) * p.splits * 2;
  float mm = -INFINITY;
  for (int s = 0; s < p.splits; ++s) mm = fmaxf(mm, pm[2 * s]);
  float ll = 0.f, oo = 0.f;
  for (int s = 0; s < p.splits; ++s) {
    const float a = mm == -INFINITY ? 0.f : __expf(pm[2 * s] - mm);
    ll += pm[2 * s + 1] * a;
    oo += p.part_o[(((int64_t)b * p.hq + h) * p.splits + s) * p.dv + d] * a;
  }
  p.o[(int64_t)row * p.so + (int64_t)h * p.dv + d] =
      from_f<T>(oo * decode_factor(p, row, h, mm, ll) * decode_gate(p, row, h, d));
}

__device__ __forceinline__ float dot8(const bf16x8& a, const bf16x8& b) {
  typedef __bf16 bf16x2 __attribute__((ext_vector_type(2)));
  float c = 0.f;
#pragma unroll
  for (int j = 0; j < 4; ++j)
    c = __builtin_amdgcn_fdot2_f32_bf16(bf16x2{a[2 * j], a[2 * j + 1]}, bf16x2{b[2 * j], b[2 * j + 1]}, c, false);
  return c;
}

template <int LPK, int GM>
__global__ __launch_bounds__(256) void paged_decode_kernel(PagedDecodeParams<bf16> p) {
  constexpr int KPW = 64 / LPK;
  constexpr int U = GM >= 8 ? 2 : 4;  // (registers)
  __shared__ float red[4][GM][2 + 8 * LPK];
  const int G = p.hq / p.hkv, gb = (G + GM - 1) / GM;
  const int split = blockIdx.x, hk = blockIdx.y / gb, g0 = (blockIdx.y % gb) * GM, b = blockIdx.z;
  const int gn = min(GM, G - g0), h0 = hk * G + g0;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int kl = lane / LPK, c = lane % LPK;
  const DecodeToken tk = decode_token(p, b);
  const DecodeKeys keys = decode_keys(p, tk.pos, split);
  const int j0 = keys.j0, j1 = keys.j1;
  const PageTable pages(p.block_tables + (int64_t)tk.seq * p.max_blocks, p.block_size, p.max_blocks);
  const int64_t kv_row = (int64_t)p.hkv * (p.dk + p.dv);
  // lanes past a head's size read its start: their q is zero, their value columns are not stored
  const bool k_on = 8 * c < p.dk, v_on = 8 * c < p.dv;
  const bf16* kbase = p.cache + (int64_t)hk * p.dk + (k_on ? c * 8 : 0);
  const bf16* vbase = p.cache + (int64_t)p.hkv * p.dk + (int64_t)hk * p.dv + (v_on ? c * 8 : 0);

  bf16x8 qv[GM];
#pragma unroll
  for (int g = 0; g < GM; ++g) {
    qv[g] = bf16x8{};
    if (g < gn && k_on)
      qv[g] = *reinterpret_cast<const bf16x8*>(p.q + (int64_t)tk.row * p.sq + (int64_t)(h0 + g) * p.dk + c * 8);
  }
  float m[GM], l[GM], acc[GM][8];
#pragma unroll
  for (int g = 0; g < GM; ++g) {
    m[g] = -INFINITY;
    l[g] = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) acc[g][e] = 0.f;
  }
  bf16x8 kn[U], vn[U];
  constexpr int STEP = 4 * KPW;  // keys between a lane group's consecutive ones
  // all block numbers, then all rows: two round trips for U keys. Keys past the end read the last one (weight zero).
  auto fetch = [&](int j) {
    int64_t r[U];
#pragma unroll
    for (int u = 0; u < U; ++u) r[u] = pages.slot(keys.pos(min(j + u * STEP, j1 - 1))) * kv_row;
#pragma unroll
    for (int u = 0; u < U; ++u) {
      kn[u] = *reinterpret_cast<const bf16x8*>(kbase + r[u]);
      vn[u] = *reinterpret_cast<const bf16x8*>(vbase + r[u]);
    }
  };
  int j = j0 + w * KPW + kl;
  fetch(j);
  for (; j - kl < j1; j += U * STEP) {
    bf16x8 kc[U], vc[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      kc[u] = kn[u];
      vc[u] = vn[u];
    }
    fetch(j + U * STEP);
#pragma unroll
    for (int g = 0; g < GM; ++g) {
      if (g >= gn) break;
      float sc[U];
#pragma unroll
      for (int u = 0; u < U; ++u) sc[u] = group_sum<LPK>(dot8(qv[g], kc[u])) * p.scale;
      if (p.softcap > 0.f) {
        const float cap2 = p.softcap * kLog2e, inv2 = 2.f / p.softcap;
#pragma unroll
        for (int u = 0; u < U; ++u) sc[u] = soft_cap2(sc[u] * kLog2e, cap2, inv2) / kLog2e;
      }
      float mn = m[g];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        sc[u] = j + u * STEP < j1 ? sc[u] : -INFINITY;
        mn = fmaxf(mn, sc[u]);
      }
      const bool none = mn == -INFINITY;
      const float a = none ? 1.f : __expf(m[g] - mn);
      l[g] *= a;
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[g][e] *= a;
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const float e_s = none ? 0.f : __expf(sc[u] - mn);
        l[g] += e_s;
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[g][e] += e_s * (float)vc[u][e];
      }
      m[g] = mn;
    }
  }
#pragma unroll
  for (int g = 0; g < GM; ++g) {
    if (g >= gn) break;
#pragma unroll
    for (int off = LPK; off < 64; off <<= 1) {
      const float mo = __shfl_xor(m[g], off, 64), lo = __shfl_xor(l[g], off, 64);
      const float mn = fmaxf(m[g], mo);
      const float a = mn == -INFINITY ? 0.f : __expf(m[g] - mn), ao = mn == -INFINITY ? 0.f : __expf(mo - mn);
      l[g] = l[g] * a + lo * ao;
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[g][e] = acc[g][e] * a + __shfl_xor(acc[g][e], off, 64) * ao;
      m[g] = mn;
    }
  }
  if (kl == 0) {
#pragma unroll
    for (int g = 0; g < GM; ++g) {
      if (g >= gn) break;
      if (c == 0) {
        red[w][g][0] = m[g];
        red[w][g][1] = l[g];
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) red[w][g][2 + c * 8 + e] = acc[g][e];
    }
  }
  __syncthreads();
  for (int t = threadIdx.x; t < gn * LPK; t += 256) {
    const int g = t / LPK, cc = t % LPK;
    float mm = -INFINITY;
    for (int ww = 0; ww < 4; ++ww) mm = fmaxf(mm, red[ww][g][0]);
    float ll = 0.f, oo[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    for (int ww = 0; ww < 4; ++ww) {
      const float a = mm == -INFINITY ? 0.f : __expf(red[ww][g][0] - mm);
      ll += red[ww][g][1] * a;
#pragma unroll
      for (int e = 0; e < 8; ++e) oo[e] += red[ww][g][2 + cc * 8 + e] * a;
    }
    const int h = h0 + g;
    if (p.splits == 1) {
      const float f = decode_factor(p, tk.row, h, mm, ll);
#pragma unroll
      for (int e = 0; e < 8; ++e) oo[e] *= f;
      if (p.gw > 1 && 8 * cc < p.dv)
#pragma unroll
        for (int e = 0; e < 8; ++e) oo[e] *= decode_gate(p, tk.row, h, 8 * cc + e);
      if (8 * cc < p.dv) Vec8<bf16>::store(p.o + (int64_t)tk.row * p.so + (int64_t)h * p.dv + cc * 8, oo);
    } else {
      const int64_t pi = ((int64_t)b * p.hq + h) * p.splits + split;
      if (8 * cc < p.dv) Vec8<float>::store(p.part_o + pi * p.dv + cc * 8, oo);
      if (cc == 0) {
        p.part_ml[2 * pi] = mm;
        p.part_ml[2 * pi + 1] = ll;
      }
    }
  }
  if (p.splits > 1 && p.counters != nullptr) {
    // release this split's partials (device scope: the splits run on every XCD), count it in; the last one in
    // acquires all of them and merges
    __shared__ int s_last;
    __threadfence();
    __syncthreads();
    if (threadIdx.x == 0) s_last = atomicAdd(p.counters + b * p.hkv + hk, 1) == p.splits - 1;
    __syncthreads();
    if (!s_last) return;
    __threadfence();
    for (int t = threadIdx.x; t < gn * p.dv; t += 256) decode_merge_splits(p, b, h0 + t / p.dv, t % p.dv, tk.row);
    if (threadIdx.x == 0) p.counters[b * p.hkv + hk] = 0;
  }
}

// any type and sizes: one workgroup per (split, query head, token); a wave's lanes share the dims of a key, then every
// thread owns output columns
constexpr int kPlainKeys = 64;

template <typename T>
__global__ __launch_bounds__(256) void paged_plain_kernel(PagedDecodeParams<T> p) {
  extern __shared__ float sm[];  // q [dk], acc [dv], scores / weights [kPlainKeys]
  float* sq = sm;
  float* acc = sm + p.dk;
  float* ss = acc + p.dv;
  const int split = blockIdx.x, h = blockIdx.y, b = blockIdx.z, hk = h / (p.hq / p.hkv);
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const DecodeToken tk = decode_token(p, b);
  const DecodeKeys keys = decode_keys(p, tk.pos, split);
  const int j0 = keys.j0, j1 = keys.j1;
  const PageTable pages(p.block_tables + (int64_t)tk.seq * p.max_blocks, p.block_size, p.max_blocks);
  const int64_t kv_row = (int64_t)p.hkv * (p.dk + p.dv);
  auto slot = [&](int j) { return p.cache + pages.slot(keys.pos(j)) * kv_row; };
  for (int i = threadIdx.x; i < p.dk; i += 256) sq[i] = to_f(p.q[(int64_t)tk.row * p.sq + (int64_t)h * p.dk + i]);
  for (int i = threadIdx.x; i < p.dv; i += 256) acc[i] = 0.f;
  __syncthreads();
  float m = -INFINITY, l = 0.f;
  for (int jb = j0; jb < j1; jb += kPlainKeys) {
    const int nk = min(kPlainKeys, j1 - jb);
    for (int k = w; k < nk; k += 4) {
      const T* kr = slot(jb + k) + (int64_t)hk * p.dk;
      float s = 0.f;
      for (int i = lane; i < p.dk; i += 64) s += sq[i] * to_f(kr[i]);
      s = wave_sum(s);
      if (lane == 0) ss[k] = p.softcap > 0.f ? soft_cap(s * p.scale, p.softcap) : s * p.scale;
    }
    __syncthreads();
    float mt = m;
    for (int k = 0; k < nk; ++k) mt = fmaxf(mt, ss[k]);
    __syncthreads();
    if ((int)threadIdx.x < nk) ss[threadIdx.x] = __expf(ss[threadIdx.x] - mt);
    __syncthreads();
    const float alpha = __expf(m - mt);  // 0 at the first tile
    m = mt;
    float sum = 0.f;
    for (int k = 0; k < nk; ++k) sum += ss[k];
    l = l * alpha + sum;
    for (int i = threadIdx.x; i < p.dv; i += 256) {
      float o = acc[i] * alpha;
      for (int k = 0; k < nk; ++k) o += ss[k] * to_f(slot(jb + k)[p.hkv * p.dk + hk * p.dv + i]);
      acc[i] = o;
    }
    __syncthreads();
  }
  const int64_t pi = ((int64_t)b * p.hq + h) * p.splits + split;
  if (p.splits == 1) {
    const float f = decode_factor(p, tk.row, h, m, l);
    for (int i = threadIdx.x; i < p.dv; i += 256)
      p.o[(int64_t)tk.row * p.so + (int64_t)h * p.dv + i] = from_f<T>(acc[i] * f * decode_gate(p, tk.row, h, i));
    return;
  }
  for (int i = threadIdx.x; i < p.dv; i += 256) p.part_o[pi * p.dv + i] = acc[i];
  if (threadIdx.x == 0) {
    p.part_ml[2 * pi] = m;
    p.part_ml[2 * pi + 1] = l;
  }
}

// One workgroup per (token, q head): the split maxima / sums are loaded once, one per thread, into LDS
// (one memory round trip instead of a dependent walk over the splits), then every thread merges its output column
// over the splits from partial-o values it requested before the barrier (splits <= 64 <= threads).
template <typename T>
__global__ __launch_bounds__(256) void paged_decode_combine_kernel(PagedDecodeParams<T> p) {
  __shared__ float s_m[64], s_l[64];
  const int bh = blockIdx.x, b = bh / p.hq, h = bh % p.hq;
  const int d0 = threadIdx.x, dl = min(d0, p.dv - 1);
  // every load is issued before the barrier: the partial-o column (its addresses need no split stat) and the output
  // row overlap the stats' round trip instead of following it
  const float* po = p.part_o + (int64_t)bh * p.splits * p.dv;
  float pov[64];
#pragma unroll
  for (int s = 0; s < 64; ++s) pov[s] = s < p.splits ? po[(int64_t)s * p.dv + dl] : 0.f;
  const int row = decode_token(p, b).row;
  const float gate0 = decode_gate(p, row, h, dl);
  const float* pm = p.part_ml + (int64_t)bh * p.splits * 2;
  if (d0 < p.splits) {
    s_m[d0] = pm[2 * d0];
    s_l[d0] = pm[2 * d0 + 1];
  }
  __syncthreads();
  float mm = -INFINITY;
  for (int s = 0; s < p.splits; ++s) mm = fmaxf(mm, s_m[s]);
  float ll = 0.f, oo = 0.f;
#pragma unroll
  for (int s = 0; s < 64; ++s) {
    if (s < p.splits) {
      const float a = mm == -INFINITY ? 0.f : __expf(s_m[s] - mm);
      ll += s_l[s] * a;
      oo += pov[s] * a;
    }
  }
  const float f = decode_factor(p, row, h, mm, ll);
  T* op = p.o + (int64_t)row * p.so + (int64_t)h * p.dv;
  if (d0 < p.dv) op[d0] = from_f<T>(oo * f * gate0);
  for (int d = d0 + blockDim.x; d < p.dv; d += blockDim.x) {  // heads wider than the workgroup
    oo = 0.f;
    for (int s = 0; s < p.splits; ++s) oo += po[(int64_t)s * p.dv + d] * (mm == -INFINITY ? 0.f : __expf(s_m[s] - mm));
    op[d] = from_f<T>(oo * f * decode_gate(p, row, h, d));
  }
}

template <typename T>
void launch_combine(const PagedDecodeParams<T>& p, int n, hipStream_t st) {
  const int threads = p.dv >= 256 ? 256 : (p.dv + 63) / 64 * 64;
  hipLaunchKernelGGL(paged_decode_combine_kernel<T>, dim3(n * p.hq), dim3(threads), 0, st, p);
}

template <int LPK>
int launch_decode(const PagedDecodeParams<bf16>& p, int n, hipStream_t st) {
  const int G = p.hq / p.hkv;
#define HDS_DEC(GM)                                                                                                 \
  hipLaunchKernelGGL((paged_decode_kernel<LPK, GM>), dim3(p.splits, p.hkv * ((G + GM - 1) / GM), n), dim3(256), 0, st, p)
  if (G == 1) HDS_DEC(1); else if (G == 2) HDS_DEC(2); else if (G <= 4) HDS_DEC(4); else HDS_DEC(8);
#undef HDS_DEC
  if (p.splits > 1 && p.counters == nullptr) launch_combine(p, n, st);
  return hipGetLastError();
}

template <typename T>
int launch_plain(const PagedDecodeParams<T>& p, int n, hipStream_t st) {
  const size_t lds = (p.dk + p.dv + kPlainKeys) * sizeof(float);
  if (lds > 64 * 1024 || p.hq > 65535) return hipErrorInvalidValue;
  hipLaunchKernelGGL(paged_plain_kernel<T>, dim3(p.splits, p.hq, n), dim3(256), lds, st, p);
  if (p.splits > 1) launch_combine(p, n, st);
  return hipGetLastError();
}

template <typename T>
int launch_head_norm(const HeadNormParams<T>& p, hipStream_t st) {
  const int64_t items = (int64_t)p.n_tok * (p.hq + 2 * p.hkv);
  const int d = p.dk > p.dv ? p.dk : p.dv;
  if (p.dk % 8 || p.dv % 8 || p.ld % 8 || d > 512 || (p.v0 != nullptr && (p.ldv0 % 8 || (uintptr_t)p.v0 % 16))) {
    hipLaunchKernelGGL(head_norm_scatter_kernel<T>, dim3((items + 3) / 4), dim3(256), 0, st, p);
    return hipGetLastError();
  }
#define HDS_HN(L) \
  hipLaunchKernelGGL((head_norm_scatter8_kernel<T, L>), dim3((items + 256 / L - 1) / (256 / L)), dim3(256), 0, st, p)
  if (d <= 64) HDS_HN(8); else if (d <= 128) HDS_HN(16); else if (d <= 256) HDS_HN(32); else HDS_HN(64);
#undef HDS_HN
  return hipGetLastError();
}

}  // namespace

#define HDS_PAGED_DIMS(X) X(32) X(48) X(64) X(80) X(96) X(112) X(128) X(160) X(192) X(256)

// rot_dim: rotary prefix (0 = the whole head); cos/sin tables are [pos][rot_dim / 2]
HDS_EXPORT int hds_kv_rope_scatter(int dtype, void* qkv, int64_t sq, void* cache, const int* tok_seq,
                                   const int* tok_pos, const int* block_tables, int max_blocks, const float* cos_t,
                                   const float* sin_t, int n_tok, int hq, int hkv, int head_dim, int rot_dim,
                                   int block_size, int rotate_q, int do_rope, hipStream_t st) {
  if (n_tok <= 0) return 0;
  const int rot = (rot_dim <= 0 || rot_dim > head_dim) ? head_dim : rot_dim;
  if (head_dim % 4 || rot % 8 || (head_dim - rot) % 4) return hipErrorInvalidValue;
  const int64_t work = (int64_t)n_tok * (hq + 2 * hkv) * (rot / 8 + (head_dim - rot) / 4);
  dim3 grid(stream_grid(work, 256, 4096)), block(256);
  if (dtype == kBF16)
    hipLaunchKernelGGL(kv_rope_scatter_kernel<bf16>, grid, block, 0, st, (bf16*)qkv, sq, (bf16*)cache, tok_seq, tok_pos,
                       block_tables, max_blocks, cos_t, sin_t, n_tok, hq, hkv, head_dim, rot, block_size, rotate_q,
                       do_rope);
  else if (dtype == kF16)
    hipLaunchKernelGGL(kv_rope_scatter_kernel<_Float16>, grid, block, 0, st, (_Float16*)qkv, sq, (_Float16*)cache,
                       tok_seq, tok_pos, block_tables, max_blocks, cos_t, sin_t, n_tok, hq, hkv, head_dim, rot,
                       block_size, rotate_q, do_rope);
  else
    return hipErrorInvalidValue;
  return hipGetLastError();
}

// q heads normed in place, k heads normed into the cache, v heads copied there; qn / kn null: no norm. v0: values
// [n_tok, hkv * dv] with row stride ldv0 of which the share *mix goes into v; null: v as it is
HDS_EXPORT int hds_head_norm_scatter(int dtype, void* qkv, int64_t ld, const float* qn, const float* kn, void* cache,
                                     const int* tok_seq, const int* tok_pos, const int* block_tables, int n_tok,
                                     int max_blocks, int block_size, int hq, int hkv, int dk, int dv, float eps,
                                     const void* v0, int64_t ldv0, const float* mix, hipStream_t st) {
  if (n_tok <= 0) return 0;
  if (hq < 1 || hkv < 1 || hq % hkv || dk < 1 || dv < 1 || ld < (int64_t)(hq + hkv) * dk + (int64_t)hkv * dv ||
      (v0 != nullptr && (mix == nullptr || ldv0 < (int64_t)hkv * dv)))
    return hipErrorInvalidValue;
  if (dtype == kBF16)
    return launch_head_norm(HeadNormParams<bf16>{(bf16*)qkv, ld, qn, kn, (bf16*)cache, tok_seq, tok_pos, block_tables,
                                                 n_tok, max_blocks, block_size, hq, hkv, dk, dv, eps, (const bf16*)v0, ldv0,
                                                 mix}, st);
  if (dtype == kF32)
    return launch_head_norm(HeadNormParams<float>{(float*)qkv, ld, qn, kn, (float*)cache, tok_seq, tok_pos,
                                                  block_tables, n_tok, max_blocks, block_size, hq, hkv, dk, dv, eps,
                                                  (const float*)v0, ldv0, mix}, st);
  return hipErrorInvalidValue;
}

// bf16 head sizes the atom kernel takes (16-B rows; the caller checks sq and the q / o alignment)
HDS_EXPORT int hds_paged_attn_supported(int dk, int dv) {
  return dk >= 8 && dv >= 8 && dk % 8 == 0 && dv % 8 == 0 && dk <= 256 && dv <= 256;
}

// atoms: device int32 [n_atoms][3]; seq_meta: device int32 [n_seqs][3]; window, chunk, keep and softcap: 0 for none; sink [hq]
// and gate [tokens, hq * gw] (gw 1 or dv) may be null
HDS_EXPORT int hds_paged_attn(const void* q, int64_t sq, const void* cache, void* o, int64_t so, const int* atoms,
                              int n_atoms, const int* seq_meta, const int* block_tables, int max_blocks,
                              int block_size, int hq, int hkv, int dk, int dv, float scale, int window, int chunk,
                              int keep, float softcap, const float* sink, const void* gate, int64_t sg, int gw, hipStream_t st) {
  if (hq < 1 || hkv < 1 || hq % hkv || sq % 8 || so % 4 || !hds_paged_attn_supported(dk, dv) || window < 0 ||
      chunk < 0 || keep < 0 || (gate != nullptr && gw != 1 && (gw != dv || sg % 4 || (uintptr_t)gate % 8)))
    return hipErrorInvalidValue;
  if (n_atoms <= 0) return 0;
  PagedParams p{(const bf16*)q, sq, (const bf16*)cache, (bf16*)o, so, atoms, seq_meta, block_tables, max_blocks,
                block_size, hq, hkv, dk, dv, scale, window, chunk, keep, softcap, sink, (const bf16*)gate, sg, gw};
#define HDS_CASE(d)                                                                                    \
  if (dk == d && dv == d) {                                                                            \
    hipLaunchKernelGGL((paged_attn_kernel<d, d, 4, false>), dim3(n_atoms), dim3(256), 0, st, p);       \
    return hipGetLastError();                                                                          \
  }
  HDS_PAGED_DIMS(HDS_CASE)
#undef HDS_CASE
#define HDS_PAD(a, b)                                                                                  \
  if (dk <= a && dv <= b) {                                                                            \
    hipLaunchKernelGGL((paged_attn_kernel<a, b, 4, true>), dim3(n_atoms), dim3(256), 0, st, p);        \
    return hipGetLastError();                                                                          \
  }
  HDS_PAD(64, 64) HDS_PAD(64, 128) HDS_PAD(64, 256) HDS_PAD(128, 64) HDS_PAD(128, 128) HDS_PAD(128, 256)
  HDS_PAD(256, 64) HDS_PAD(256, 128) HDS_PAD(256, 256)
#undef HDS_PAD
  return hipErrorInvalidValue;
}

HDS_EXPORT int hds_paged_rows_per_atom() { return 128; }

// the vectorised single-token kernel (bf16): any group size, head sizes that are multiples of 8 up to 256
HDS_EXPORT int hds_paged_decode_supported(int dk, int dv) { return hds_paged_attn_supported(dk, dv); }

// key splits for n_seqs sequences of at most max_ctx keys: >= 2 workgroups per CU overall, >= 32 keys per split
HDS_EXPORT int hds_paged_decode_splits(int n_seqs, int hkv, int max_ctx) {
  const int groups = n_seqs * hkv;
  int splits = (512 + groups - 1) / groups;
  const int by_len = (max_ctx + 31) / 32;
  splits = splits < by_len ? splits : by_len;
  return splits < 1 ? 1 : (splits > 64 ? 64 : splits);
}

// Single tokens. seq_meta: one sequence with one new token each (n of them); null: the n tokens toks (null: 0 .. n - 1)
// of a step described by tok_seq / tok_pos. plain: the kernel for any type and size (always for float32).
// counters: null -> the splits are merged by a second (combine) launch; else n * hkv zeroed ints and the last
// workgroup of each (token, kv head) merges them in the same launch (at most kDecGMax query heads per kv head)
HDS_EXPORT int hds_paged_decode(int dtype, int plain, const void* q, int64_t sq, const void* cache, void* o, int64_t so,
                                float* part_o, float* part_ml, const int* seq_meta, const int* toks,
                                const int* tok_seq, const int* tok_pos, const int* block_tables, int max_blocks,
                                int block_size, int n, int hq, int hkv, int dk, int dv, int splits, float scale,
                                int window, int chunk, int keep, float softcap, const float* sink, const void* gate,
                                int64_t sg, int gw, int* counters, hipStream_t st) {
  if (n <= 0) return 0;
  if (hq < 1 || hkv < 1 || hq % hkv || dk < 1 || dv < 1 || splits < 1 || splits > 64 || n > 65535 ||
      window < 0 || chunk < 0 || keep < 0 || (gate != nullptr && gw != 1 && gw != dv) ||
      (seq_meta == nullptr && (tok_seq == nullptr || tok_pos == nullptr)) ||
      (splits > 1 && (!part_o || !part_ml)))  // <= 64: the combine kernel stages the split stats in LDS
    return hipErrorInvalidValue;
  if (dtype == kF32) {
    return launch_plain(PagedDecodeParams<float>{(const float*)q, sq, (const float*)cache, (float*)o, so, part_o,
                                                 part_ml, seq_meta, toks, tok_seq, tok_pos, block_tables, max_blocks,
                                                 block_size, hq, hkv, dk, dv, splits, scale, window, chunk, keep, softcap,
                                                 sink, (const float*)gate, sg, gw, nullptr}, n, st);
  }
  if (dtype != kBF16) return hipErrorInvalidValue;
  PagedDecodeParams<bf16> p{(const bf16*)q, sq, (const bf16*)cache, (bf16*)o, so, part_o, part_ml, seq_meta, toks,
                            tok_seq, tok_pos, block_tables, max_blocks, block_size, hq, hkv, dk, dv, splits, scale,
                            window, chunk, keep, softcap, sink, (const bf16*)gate, sg, gw, counters};
  if (plain) {
    p.counters = nullptr;
    return launch_plain(p, n, st);
  }
  if (!hds_paged_decode_supported(dk, dv) || sq % 8 || so % 8 || hkv > 65535 / kDecGMax ||
      (counters != nullptr && hq / hkv > kDecGMax))
    return hipErrorInvalidValue;
  const int d = dk > dv ? dk : dv;
  if (d <= 32) return launch_decode<4>(p, n, st);
  if (d <= 64) return launch_decode<8>(p, n, st);
  if (d <= 128) return launch_decode<16>(p, n, st);
  return launch_decode<32>(p, n, st);
}
