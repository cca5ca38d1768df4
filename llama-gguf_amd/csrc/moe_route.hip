// moe_route.hip — a block's tokens to their experts (layered.h): the largest scores of every token, then the (token, expert) pairs grouped
// by expert for the grouped products.  Where a pair lies within its group has no influence on any result.
#include "layered.h"
#include "layered_device.h"

namespace lgh {

__global__ void __launch_bounds__(256) moe_topk_kernel(const MoeRoute a) {
  __shared__ __attribute__((aligned(16))) float z[kMaxExperts];
  const uint32_t t = blockIdx.x, ep = (a.experts + 3) & ~3u;
  for (uint32_t e = threadIdx.x; e < ep; e += 256) z[e] = e < a.experts ? rank_key(a.logits[(size_t)t * a.ldl + e]) : -INFINITY;
  __syncthreads();
  rank_experts(z, a.experts, a.top, a.sel + (size_t)t * a.top, a.w + (size_t)t * a.top);
}

// one workgroup: sizes of the groups, their first rows and row tiles, then a row for every pair
__global__ void __launch_bounds__(1024) moe_group_rows_kernel(const MoeRoute a) {
  __shared__ int cnt[kMaxExperts], row0[kMaxExperts], tile0[kMaxExperts];
  const uint32_t tid = threadIdx.x, pairs = a.M * a.top;
  cnt[tid] = 0;
  __syncthreads();
  for (uint32_t p = tid; p < pairs; p += 1024) atomicAdd(&cnt[a.sel[p]], 1);
  __syncthreads();
  const int n = cnt[tid], nt = (n + (int)a.bm - 1) / (int)a.bm;
  row0[tid] = n;
  tile0[tid] = nt;
  __syncthreads();
  for (uint32_t d = 1; d < kMaxExperts; d *= 2) {   // running sums
    const int r = tid >= d ? row0[tid - d] : 0, k = tid >= d ? tile0[tid - d] : 0;
    __syncthreads();
    row0[tid] += r;
    tile0[tid] += k;
    __syncthreads();
  }
  const int first = row0[tid] - n, tfirst = tile0[tid] - nt;
  const uint32_t used = (uint32_t)tile0[kMaxExperts - 1];
  if (tid < a.experts) {
    a.seg[tid] = first;
    if (tid + 1 == a.experts) a.seg[a.experts] = first + n;
    for (int i = 0; i < nt; i++) {
      a.tile_e[tfirst + i] = (int)tid;
      a.tile_row[tfirst + i] = first + i * (int)a.bm;
    }
  }
  for (uint32_t i = used + tid; i < a.tiles; i += 1024) { a.tile_e[i] = -1; a.tile_row[i] = 0; }
  cnt[tid] = first;
  __syncthreads();
  for (uint32_t p = tid; p < pairs; p += 1024) {
    const int r = atomicAdd(&cnt[a.sel[p]], 1);
    a.slot[p] = r;
    a.src[r] = (int)(p / a.top);
    a.roww[r] = a.w[p];
  }
}

uint32_t moe_max_tiles(uint32_t rows, uint32_t experts, uint32_t bm) { return rows / bm + (rows < experts ? rows : experts); }

hipError_t moe_route_launch(const MoeRoute& a, hipStream_t st) {
  static_assert(kMaxExperts == 1024, "one thread per expert");
  if (a.M == 0 || a.top == 0 || a.top > a.experts || a.top > kMaxTop || a.experts > kMaxExperts || a.bm == 0 || a.tiles < moe_max_tiles(a.M * a.top, a.experts, a.bm))
    return hipErrorInvalidValue;
  hipLaunchKernelGGL(moe_topk_kernel, dim3(a.M), dim3(256), 0, st, a);
  hipLaunchKernelGGL(moe_group_rows_kernel, dim3(1), dim3(1024), 0, st, a);
  return hipGetLastError();
}

}  // namespace lgh
