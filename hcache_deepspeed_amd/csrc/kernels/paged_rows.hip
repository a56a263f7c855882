// Rows of a paged cache <-> plain matrices: gathered prefixes, HCache latents out of the pages and back.
#include "hds_common.h"

namespace {
using namespace hds;

// rows between the pages and a plain [n, W] matrix (ld elements a row); dst_row null: row i
template <typename T, bool TO_CACHE>
__global__ __launch_bounds__(256) void paged_rows_kernel(T* __restrict__ cache, T* __restrict__ rows, int64_t ld,
                                                          const int* __restrict__ seq, const int* __restrict__ pos,
                                                          const int* __restrict__ dst_row,
                                                          const int* __restrict__ tables, int max_blocks,
                                                          int block_size, int W, int n) {
  const int i = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (i >= n) return;
  const int p = pos[i];
  T* c = cache + ((int64_t)tables[(int64_t)seq[i] * max_blocks + p / block_size] * block_size + p % block_size) * W;
  T* r = rows + (int64_t)(dst_row != nullptr ? dst_row[i] : i) * ld;
  constexpr int V = 16 / sizeof(T);
  if (W % V == 0 && ((uintptr_t)rows | (uintptr_t)(ld * sizeof(T))) % 16 == 0) {
    const u32x4* src = reinterpret_cast<const u32x4*>(TO_CACHE ? r : c);
    u32x4* dst = reinterpret_cast<u32x4*>(TO_CACHE ? c : r);
    for (int k = lane; k < W / V; k += 64) dst[k] = src[k];
    return;
  }
  for (int k = lane; k < W; k += 64) {
    if (TO_CACHE) c[k] = r[k]; else r[k] = c[k];
  }
}

}  // namespace

HDS_EXPORT int hds_paged_rows(int dtype, int to_cache, void* cache, void* rows, int64_t ld, const int* seq,
                               const int* pos, const int* dst_row, const int* tables, int max_blocks, int block_size,
                               int W, int n, hipStream_t st) {
  if (n <= 0) return 0;
  if (W < 1 || ld < W || block_size < 1) return hipErrorInvalidValue;
#define HDS_PR(TT, CC)                                                                                              \
  hipLaunchKernelGGL((paged_rows_kernel<TT, CC>), dim3((n + 3) / 4), dim3(256), 0, st, (TT*)cache, (TT*)rows, ld, \
                     seq, pos, dst_row, tables, max_blocks, block_size, W, n)
  if (dtype == kBF16) {
    if (to_cache) HDS_PR(bf16, true); else HDS_PR(bf16, false);
  } else if (dtype == kF32) {
    if (to_cache) HDS_PR(float, true); else HDS_PR(float, false);
  } else {
    return hipErrorInvalidValue;
  }
#undef HDS_PR
  return hipGetLastError();
}
