// Grouped (MoE) GEMM for gfx950: for every expert e, Y[o_e : o_{e+1}] = X[o_e : o_{e+1}] . W[e]^T
// with X [T, K] expert-contiguous rows (the permuted token order), W [E, N, K] (nn.Linear layout) and
// o = exclusive prefix of the per-expert row counts, kept ON THE DEVICE (no host sync on the routing).
//
// Reference parity: SURVEY.md §2.10 N15 / §2.11 K37 — the CUTLASS grouped MoE GEMM of
// inference/v2/kernels/cutlass_ops/moe_gemm (external libdeepspeedft). Not a translation: one launch covers
// every expert's ragged row block, no capacity padding (dropless), and the tile schedule is built on the GPU.
//
// Design (cdna_hip_programming.md §3/§5):
//   * a tiny planning kernel turns the device offsets into a tile list (expert, m0) and a tile count;
//     the GEMM grid is the host-side upper bound ceil(T/128)+E, blocks past the count exit at once;
//   * 128(N) x 128(tokens) block tile, BK = 128, 4 waves each owning a 64 x 64 quadrant = 2 x 2
//     v_mfma_f32_32x32x16_bf16 accumulators. Operand orientation D = W . X^T puts the token on the lane
//     and 4 consecutive output features in consecutive accumulator registers, so the epilogue writes
//     8-byte bf16x4 vectors of one output row;
//   * both operands are K-contiguous, staged by LDS-DMA (global_load_lds_dwordx4) into the XOR-swizzled
//     64 x 256 B tiles of attn_common.h (conflict-free ds_read_b128 A/B fragments), double-buffered:
//     the next K tile streams in while the current one feeds the MFMAs;
//   * options (serving, hds_experts_gemm): X rows read through an index list instead of being permuted first; W = [gate;
//     up] with the activation silu(gate) * up or the clamped unit, optionally after a factor per row, in the epilogue -- a
//     wave then holds the accumulators of the same features of both halves; a tile list made elsewhere (experts.hip);
//   * blockIdx.x walks N tiles fastest so the (consecutively dispatched, XCD-round-robin) blocks of one
//     token tile share the X tile in L2 while W[e] streams.
#include "attn_common.h"

using namespace hds;
using namespace hds::attn;

namespace {

constexpr int BM = 128;  // tokens per block tile
constexpr int BN = 128;  // output features per block tile
constexpr int BK = 128;  // reduction depth per stage (one 256-byte bf16 row per tile row)

template <int TM>
__global__ __launch_bounds__(64) void gg_plan_kernel(const int* __restrict__ offs, int E, int T,
                                                     int* __restrict__ tile_e, int* __restrict__ tile_m,
                                                     int* __restrict__ n_tiles, int max_tiles) {
  // single wave: serial prefix over experts (E <= a few hundred), lanes fill each expert's tiles
  const int lane = threadIdx.x;
  int base = 0;
  for (int e = 0; e < E; ++e) {
    const int lo = min(max(offs[e], 0), T), hi = min(max(offs[e + 1], lo), T);  // never trust offsets
    const int t = (hi - lo + TM - 1) / TM;
    for (int i = lane; i < t; i += 64) {
      if (base + i < max_tiles) {
        tile_e[base + i] = e;
        tile_m[base + i] = i * TM;
      }
    }
    base += t;
  }
  if (lane == 0) *n_tiles = base < max_tiles ? base : max_tiles;
}

// epilogue of gate | up products
struct GatedUnit {
  const float* weight;  // [rows] or null
  int clamped;
  float limit;
  __device__ __forceinline__ float factor(int row) const { return weight != nullptr ? weight[row] : 1.f; }
  __device__ __forceinline__ float operator()(float g, float u, float w) const {
    g *= w;
    u *= w;
    if (!clamped) return g / (1.f + __expf(-g)) * u;
    g = fminf(g, limit);
    return g / (1.f + __expf(-1.702f * g)) * (fminf(fmaxf(u, -limit), limit) + 1.f);
  }
};

// GATHER: row r of the sorted order is x[src[r]] (n_src rows of x). GLU: w holds 2N rows per expert, gate then up.
template <bool GATHER, bool GLU>
__global__ __launch_bounds__(256) void gg_kernel(const bf16* __restrict__ x, int64_t ldx,
                                                 const int* __restrict__ src, int n_src, const bf16* __restrict__ w,
                                                 bf16* __restrict__ y, const int* __restrict__ offs,
                                                 const int* __restrict__ tile_e, const int* __restrict__ tile_m,
                                                 const int* __restrict__ n_tiles, int T, int N, int K, int ldy,
                                                 GatedUnit unit) {
  const int t = blockIdx.y;
  if (t >= *n_tiles) return;  // block-uniform exit before any barrier
  const int e = tile_e[t];
  const int m0 = tile_m[t];
  const int row0 = min(max(offs[e], 0), T);
  const int rows = min(max(offs[e + 1], row0), T) - row0;  // >= 1: the plan only emits tiles of non-empty experts
  const int n0 = blockIdx.x * (GLU ? BN / 2 : BN);

  __shared__ __attribute__((aligned(16))) char smem[2 * 65536];
  __shared__ int s_src[GATHER ? BM : 1];
  // buffer b: W tile halves at [b*64K, +16K, ...], X tile halves at [b*64K + 32K, +16K]
  const bf16* wb = w + (int64_t)e * (GLU ? 2 : 1) * N * K + (int64_t)n0 * K;
  const int64_t whalf = (int64_t)(GLU ? N : 64) * K;  // second half of the W tile: the up rows, or the next 64 rows
  const bf16* xb = x + (int64_t)row0 * ldx;
  if constexpr (GATHER) {
    for (int r = threadIdx.x; r < BM; r += 256)
      s_src[r] = min(max(src[row0 + min(m0 + r, rows - 1)], 0), n_src - 1);
    __syncthreads();
  }
  auto wrow = [&](int half, int kt) {
    return [=](int r) { return wb + half * whalf + (int64_t)r * K + (int64_t)kt * BK; };
  };
  auto xrow = [&](int half, int kt) {
    const int* sp = s_src;
    return [=](int r) {
      if constexpr (GATHER) {
        return x + (int64_t)sp[64 * half + r] * ldx + (int64_t)kt * BK;
      } else {
        int m = m0 + 64 * half + r;
        m = m < rows ? m : rows - 1;
        return xb + (int64_t)m * ldx + (int64_t)kt * BK;
      }
    };
  };
  auto stage = [&](int buf, int kt) {
    char* s = smem + buf * 65536;
    stage_tile64<4>(s, wrow(0, kt));
    stage_tile64<4>(s + 16384, wrow(1, kt));
    stage_tile64<4>(s + 32768, xrow(0, kt));
    stage_tile64<4>(s + 49152, xrow(1, kt));
  };

  const int wv = threadIdx.x >> 6;
  const int wn = wv & 1, wm = wv >> 1;
  f32x16 acc[2][2];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) acc[i][j] = f32x16{};

  const int KT = K / BK;
  stage(0, 0);
  __syncthreads();
  for (int kt = 0; kt < KT; ++kt) {
    const int buf = kt & 1;
    if (kt + 1 < KT) stage(buf ^ 1, kt + 1);
    // GLU: the wave's two row blocks are the same 32 features of the gate and of the up half
    const char* Wt = smem + buf * 65536 + (GLU ? 0 : wn * 16384);
    const char* Xt = smem + buf * 65536 + 32768 + wm * 16384;
#pragma unroll
    for (int ks = 0; ks < 8; ++ks) {
      const bf16x8 a0 = read_rows(Wt, GLU ? 32 * wn : 0, ks);
      const bf16x8 a1 = GLU ? read_rows(Wt + 16384, 32 * wn, ks) : read_rows(Wt, 32, ks);
      const bf16x8 b0 = read_rows(Xt, 0, ks), b1 = read_rows(Xt, 32, ks);
      acc[0][0] = mfma(a0, b0, acc[0][0]);
      acc[0][1] = mfma(a0, b1, acc[0][1]);
      acc[1][0] = mfma(a1, b0, acc[1][0]);
      acc[1][1] = mfma(a1, b1, acc[1][1]);
    }
    __syncthreads();
  }

  // epilogue: lane = token, registers 4g..4g+3 = 4 consecutive output features
  const int lane = threadIdx.x & 63;
  const int h = lane >> 5;
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int m = m0 + 64 * wm + 32 * j + (lane & 31);
    if (m >= rows) continue;
    bf16* yr = y + (int64_t)(row0 + m) * ldy + n0 + (GLU ? 32 : 64) * wn;
    if constexpr (GLU) {
      const float rw = unit.factor(row0 + m);
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        bf16x4 v;
#pragma unroll
        for (int q = 0; q < 4; ++q) v[q] = (bf16)unit(acc[0][j][4 * g + q], acc[1][j][4 * g + q], rw);
        *reinterpret_cast<bf16x4*>(yr + acc_row(4 * g, h)) = v;
      }
      continue;
    }
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        bf16x4 v;
#pragma unroll
        for (int q = 0; q < 4; ++q) v[q] = (bf16)acc[i][j][4 * g + q];
        *reinterpret_cast<bf16x4*>(yr + 32 * i + acc_row(4 * g, h)) = v;
      }
  }
}

// ---------------------------------------------------------------------------------------------------------------
// Large-expert variant: 256 x 256 block tile, BK = 64, 8 waves (2 along N x 4 along tokens, 128 x 64 per wave =
// 4 x 2 accumulators). The per-wave tile halves the LDS bytes per MFMA of the 128^2 kernel (6 ds_read_b128 per
// 8 MFMA instead of 4 per 4), which is what bounds the small tile. LDS: two buffers of (256 + 256) rows x 128 B
// = 128 KB; rows of 128 B use the XOR swizzle chunk ^ ((row >> 1) & 7): a 16-lane ds_read_b128 group reading 16
// consecutive rows at one logical chunk hits 16 distinct 16-B bank slots (row & 1 selects the half of the
// 256-B bank line). Staging is LDS-DMA (lane-linear destination, swizzle applied to the source address).
// Blocks are remapped so each XCD works on a contiguous range of (token tile, N tile) pairs, rastered in groups of
// 4 token tiles so co-resident blocks share X and W panels in the same L2.
// ---------------------------------------------------------------------------------------------------------------
constexpr int BM2 = 256, BN2 = 256, BK2 = 64;

__device__ __forceinline__ int off128(int row, int ch) { return row * 128 + 16 * (ch ^ ((row >> 1) & 7)); }

// stage `rows` x 128 B (rows % 64 == 0) with an NW-wave block: one wave-instruction fills 8 rows
template <int NW, int ROWS, typename RowPtr>
__device__ __forceinline__ void stage128(char* lds, RowPtr row_ptr) {
  const int lane = threadIdx.x & 63;
  const int w = threadIdx.x >> 6;
  constexpr int PER = ROWS / 8 / NW;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int n = w * PER + i;
    const int row = 8 * n + (lane >> 3);
    const int ch = (lane & 7) ^ ((row >> 1) & 7);
    const char* src = (const char*)row_ptr(row) + ch * 16;
    __builtin_amdgcn_global_load_lds((gbl_void*)src, (lds_void*)(lds + n * 1024), 16, 0, 0);
  }
}

__device__ __forceinline__ bf16x8 frag128(const char* lds, int row0, int ks) {
  const int lane = threadIdx.x & 63;
  return *reinterpret_cast<const bf16x8*>(lds + off128(row0 + (lane & 31), 2 * ks + (lane >> 5)));
}

template <bool GATHER, bool GLU>
__global__ __launch_bounds__(512) void gg_big_kernel(const bf16* __restrict__ x, int64_t ldx,
                                                     const int* __restrict__ src, int n_src,
                                                     const bf16* __restrict__ w, bf16* __restrict__ y, const int* __restrict__ offs,
                                                     const int* __restrict__ tile_e, const int* __restrict__ tile_m,
                                                     const int* __restrict__ n_tiles, int T, int N, int K, int ldy,
                                                     int ntn, GatedUnit unit) {
  // XCD-contiguous remap of the 1-D grid (bijective for any size)
  const int nwg = gridDim.x, orig = blockIdx.x;
  const int q = nwg / 8, r = nwg % 8, xcd = orig % 8;
  const int id = (xcd < r ? xcd * (q + 1) : r * (q + 1) + (xcd - r) * q) + orig / 8;
  // grouped raster: consecutive ids sweep GT token tiles before moving to the next N tile, so the ~32 blocks an
  // XCD runs at once cover a GT x (32/GT) rectangle and share both X and W K-slices in its L2
  constexpr int GT = 4;
  const int mt = gridDim.x / ntn;  // token-tile slots (host upper bound)
  const int grp = id / (GT * ntn), rem = id % (GT * ntn);
  const int gsz = min(GT, mt - grp * GT);
  const int t = grp * GT + rem % gsz;
  if (t >= *n_tiles) return;  // block-uniform exit before any barrier
  const int n0 = (rem / gsz) * (GLU ? BN2 / 2 : BN2);
  const int e = tile_e[t];
  const int m0 = tile_m[t];
  const int row0 = min(max(offs[e], 0), T);
  const int rows = min(max(offs[e + 1], row0), T) - row0;

  __shared__ __attribute__((aligned(16))) char smem[2 * 65536];  // [buf][W 32 KB | X 32 KB]
  __shared__ int s_src[GATHER ? BM2 : 1];
  const bf16* wb = w + (int64_t)e * (GLU ? 2 : 1) * N * K + (int64_t)n0 * K;
  const bf16* xb = x + (int64_t)row0 * ldx;
  if constexpr (GATHER) {
    if (threadIdx.x < BM2)
      s_src[threadIdx.x] = min(max(src[row0 + min(m0 + (int)threadIdx.x, rows - 1)], 0), n_src - 1);
    __syncthreads();
  }
  auto stage = [&](int buf, int kt) {
    char* s = smem + buf * 65536;
    const int64_t k0 = (int64_t)kt * BK2;
    const int* sp = s_src;
    // GLU: tile rows 0-127 are gate features, 128-255 the same features of the up half
    const int64_t up = GLU ? (int64_t)(N - 128) * K : 0;
    stage128<8, 256>(s, [=](int rr) { return wb + (int64_t)rr * K + k0 + (GLU && rr >= 128 ? up : 0); });
    stage128<8, 256>(s + 32768, [=](int rr) {
      if constexpr (GATHER) {
        return x + (int64_t)sp[rr] * ldx + k0;
      } else {
        int m = m0 + rr;
        m = m < rows ? m : rows - 1;
        return xb + (int64_t)m * ldx + k0;
      }
    });
  };

  const int wv = threadIdx.x >> 6;
  const int wn = wv & 1, wm = wv >> 1;  // 128 features x 64 tokens per wave
  f32x16 acc[4][2];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) acc[i][j] = f32x16{};

  const int KT = K / BK2;
  stage(0, 0);
  __syncthreads();
  for (int kt = 0; kt < KT; ++kt) {
    const int buf = kt & 1;
    if (kt + 1 < KT) stage(buf ^ 1, kt + 1);
    const char* Wt = smem + buf * 65536 + wn * (GLU ? 64 : 128) * 128;
    const char* Xt = smem + buf * 65536 + 32768 + wm * 64 * 128;
#pragma unroll
    for (int ks = 0; ks < 4; ++ks) {
      bf16x8 a[4], b[2];
#pragma unroll
      for (int i = 0; i < 4; ++i) a[i] = frag128(Wt, GLU ? 32 * (i & 1) + 128 * (i >> 1) : 32 * i, ks);
#pragma unroll
      for (int j = 0; j < 2; ++j) b[j] = frag128(Xt, 32 * j, ks);
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i][j] = mfma(a[i], b[j], acc[i][j]);
    }
    __syncthreads();
  }

  const int lane = threadIdx.x & 63;
  const int h = lane >> 5;
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int m = m0 + 64 * wm + 32 * j + (lane & 31);
    if (m >= rows) continue;
    bf16* yr = y + (int64_t)(row0 + m) * ldy + n0 + (GLU ? 64 : 128) * wn;
    if constexpr (GLU) {
      const float rw = unit.factor(row0 + m);
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int g = 0; g < 4; ++g) {
          bf16x4 v;
#pragma unroll
          for (int q = 0; q < 4; ++q) v[q] = (bf16)unit(acc[i][j][4 * g + q], acc[i + 2][j][4 * g + q], rw);
          *reinterpret_cast<bf16x4*>(yr + 32 * i + acc_row(4 * g, h)) = v;
        }
      continue;
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        bf16x4 v;
#pragma unroll
        for (int qq = 0; qq < 4; ++qq) v[qq] = (bf16)acc[i][j][4 * g + qq];
        *reinterpret_cast<bf16x4*>(yr + 32 * i + acc_row(4 * g, h)) = v;
      }
  }
}

}  // namespace

// Upper bound of the tile count for T rows over E experts (host-side grid size / scratch sizing).
HDS_EXPORT int hds_grouped_gemm_max_tiles(int T, int E) { return (T + BM - 1) / BM + E; }

// Y [T, ldy>=N] = per-expert X . W[e]^T.  x [T, K], w [E, N, K], offs [E+1] (device, int32),
// work = int32 scratch of 2*hds_grouped_gemm_max_tiles(T, E) + 1 elements. Requires N % 128 == 0, K % 128 == 0.
// variant: 0 = auto (256^2 tiles when N % 256 == 0 and the average expert has >= 256 rows), 1 = 128^2, 2 = 256^2.
HDS_EXPORT int hds_grouped_gemm(const void* x, const void* w, void* y, const int* offs, int* work, int T, int N, int K,
                                int E, int ldy, int variant, hipStream_t st) {
  if (T <= 0 || E <= 0) return 0;
  if (N % BN || K % BK || ldy < N || ldy % 8) return hipErrorInvalidValue;
  bool big = variant == 2 || (variant == 0 && N % BN2 == 0 && T >= BM2 * E);
  if (big && N % BN2) return hipErrorInvalidValue;
  const int cap = hds_grouped_gemm_max_tiles(T, E);
  int* tile_e = work;
  int* tile_m = work + cap;
  int* n_tiles = work + 2 * cap;
  if (big) {
    const int max_tiles = (T + BM2 - 1) / BM2 + E;  // <= cap
    const int ntn = N / BN2;
    hipLaunchKernelGGL(gg_plan_kernel<BM2>, dim3(1), dim3(64), 0, st, offs, E, T, tile_e, tile_m, n_tiles, max_tiles);
    hipLaunchKernelGGL((gg_big_kernel<false, false>), dim3(ntn * max_tiles), dim3(512), 0, st, (const bf16*)x, K,
                       (const int*)nullptr, 0, (const bf16*)w, (bf16*)y, offs, tile_e, tile_m, n_tiles, T, N, K, ldy, ntn,
                       GatedUnit{});
  } else {
    hipLaunchKernelGGL(gg_plan_kernel<BM>, dim3(1), dim3(64), 0, st, offs, E, T, tile_e, tile_m, n_tiles, cap);
    hipLaunchKernelGGL((gg_kernel<false, false>), dim3(N / BN, cap), dim3(256), 0, st, (const bf16*)x, K,
                       (const int*)nullptr, 0, (const bf16*)w, (bf16*)y, offs, tile_e, tile_m, n_tiles, T, N, K, ldy, GatedUnit{});
  }
  return hipGetLastError();
}

// Rows of a tile for T rows over E experts and N columns (what hds_experts_gemm wants its tile list to be made for)
HDS_EXPORT int hds_experts_gemm_tile(int T, int N, int E) { return N % BN2 == 0 && T >= BM2 * E ? BM2 : BM; }

// Grouped product of sorted rows with a ready tile list (tm = 128 or 256 rows, see hds_experts_gemm_tile; at most
// max_tiles entries, the number on the device). src: row of x [n_src, ldx] for every sorted row, or null: x is sorted.
// glu: w [E, 2N, K] is gate rows then up rows and y = silu(gate) * up, or the clamped unit with its limit (act 5); weight [T]
// or null multiplies the sorted rows' products in front of it. T: upper bound of the rows. K % 128 == 0; N a
// multiple of the tile's columns (128, 256; half of that with glu).
HDS_EXPORT int hds_experts_gemm(const void* x, int64_t ldx, const int* src, int n_src, const void* w, void* y, int ldy,
                                const int* offs, const int* tile_e, const int* tile_m, const int* n_tiles,
                                int max_tiles, int tm, int T, int N, int K, int E, int glu, int act, float limit,
                                const float* weight, hipStream_t st) {
  if (T <= 0 || E <= 0) return 0;
  const GatedUnit unit{weight, act == 5, limit};
  const int cols = (tm == BM2 ? BN2 : BN) / (glu ? 2 : 1);
  if ((tm != BM && tm != BM2) || N % cols || K % BK || ldx < K || ldx % 8 || ldy < N || ldy % 8 || max_tiles < 1 ||
      max_tiles > 65535 || (src != nullptr && n_src < 1) || (act != 0 && act != 5))
    return hipErrorInvalidValue;
#define HDS_EG(GA, GL)                                                                                               \
  if (tm == BM2)                                                                                                     \
    hipLaunchKernelGGL((gg_big_kernel<GA, GL>), dim3(N / cols * max_tiles), dim3(512), 0, st, (const bf16*)x, ldx,  \
                       src, n_src, (const bf16*)w, (bf16*)y, offs, tile_e, tile_m, n_tiles, T, N, K, ldy, N / cols, unit); \
  else                                                                                                               \
    hipLaunchKernelGGL((gg_kernel<GA, GL>), dim3(N / cols, max_tiles), dim3(256), 0, st, (const bf16*)x, ldx, src,  \
                       n_src, (const bf16*)w, (bf16*)y, offs, tile_e, tile_m, n_tiles, T, N, K, ldy, unit)
  if (src != nullptr) {
    if (glu) { HDS_EG(true, true); } else { HDS_EG(true, false); }
  } else {
    if (glu) { HDS_EG(false, true); } else { HDS_EG(false, false); }
  }
#undef HDS_EG
  return hipGetLastError();
}
