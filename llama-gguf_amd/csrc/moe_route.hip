// moe_route.hip — a block's tokens to their experts (layered.h): the largest scores of every token, then the (token, expert) pairs grouped
// by expert for the grouped products.  Where a pair lies within its group has no influence on any result.
#include "layered.h"
#include "layered_device.h"

namespace lgh {

// Router logits of 16 tokens and their largest scores.  8 waves share the columns; kRouteTiles * 16 experts at a time (the weights are the A operand: a
// lane ends up with 4 consecutive experts of one token), partial sums meet in LDS.
constexpr uint32_t kRouteTokens = 16, kRouteWaves = 8;

template <class T, uint32_t kRouteTiles>
__global__ void __launch_bounds__(512) moe_topk_kernel(const MoeRoute a) {
  __shared__ float red[kRouteWaves][kRouteTiles * 16][kRouteTokens];
  extern __shared__ __attribute__((aligned(16))) float z[];   // [tokens][ep]
  const uint32_t tid = threadIdx.x, lane = tid & 63, wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6)), r16 = lane & 15, g = lane >> 4;
  const uint32_t ne = a.experts + a.route.identity, t0 = blockIdx.x * kRouteTokens, ep = (ne + 3) & ~3u, m = t0 + r16 < a.M ? t0 + r16 : a.M - 1;
  const T* x = reinterpret_cast<const T*>(a.x) + (size_t)m * a.ldx + g * Frag<T>::PER;
  for (uint32_t e0 = 0; e0 < ne; e0 += kRouteTiles * 16) {
    f32x4 acc[kRouteTiles];
    const uint16_t* w[kRouteTiles];
#pragma unroll
    for (uint32_t n = 0; n < kRouteTiles; n++) {
      acc[n] = (f32x4)(0.0f);
      const uint32_t row = e0 + n * 16 + r16;
      w[n] = a.router + (size_t)(row < ne ? row : ne - 1) * a.kp + g * Frag<T>::PER;
    }
#pragma unroll (kRouteTiles == 1 ? 8 : 4)
    for (uint32_t k = wave * Frag<T>::KU; k < a.kp; k += kRouteWaves * Frag<T>::KU) {
      const typename Frag<T>::V xf = Frag<T>::load(x + k);
#pragma unroll
      for (uint32_t n = 0; n < kRouteTiles; n++) {
        typename Frag<T>::V wf;
        if constexpr (sizeof(T) == 2) {
          wf = *reinterpret_cast<const bf16x8*>(w[n] + k);
        } else {
          const u32x2 h = *reinterpret_cast<const u32x2*>(w[n] + k);
          wf.x = bf_lo(h.x); wf.y = bf_hi(h.x); wf.z = bf_lo(h.y); wf.w = bf_hi(h.y);
        }
        acc[n] = Frag<T>::mma(wf, xf, acc[n]);
      }
    }
#pragma unroll
    for (uint32_t n = 0; n < kRouteTiles; n++)
#pragma unroll
      for (uint32_t e = 0; e < 4; e++) red[wave][n * 16 + g * 4 + e][r16] = acc[n][e];
    __syncthreads();
    for (uint32_t i = tid; i < kRouteTiles * 16 * kRouteTokens; i += 512) {
      const uint32_t e = i / kRouteTokens, t = i % kRouteTokens;
      float v = 0.0f;
#pragma unroll
      for (uint32_t k = 0; k < kRouteWaves; k++) v += red[k][e][t];
      if (e0 + e < ep) z[t * ep + e0 + e] = e0 + e < ne ? rank_key(v) : -INFINITY;
    }
    __syncthreads();
  }
  if (a.route.form == LGH_ROUTER_SOFTMAX_GROUPS) {
    float* c = z + kRouteTokens * ep;
    float* gm = c + kRouteTokens * ep;
    int* sel = reinterpret_cast<int*>(gm + kRouteTokens * a.route.groups);
    float* w = reinterpret_cast<float*>(sel + kRouteTokens * a.top);
    route_groups(z, c, gm, kRouteTokens, ne, ep, a.top, a.route, sel, w);
    for (uint32_t i = tid; i < kRouteTokens * a.top; i += 512)
      if (t0 + i / a.top < a.M) { a.sel[(size_t)t0 * a.top + i] = sel[i]; a.w[(size_t)t0 * a.top + i] = w[i]; }
    return;
  }
  for (uint32_t i = tid; i < kRouteTokens * a.experts; i += 512) {
    const uint32_t t = i / a.experts;
    if (t0 + t < a.M) rank_expert(z + t * ep, a.experts, a.top, i % a.experts, a.sel + (size_t)(t0 + t) * a.top, a.w + (size_t)(t0 + t) * a.top);
  }
}

// one workgroup: sizes of the groups, their first rows and row tiles, then a row for every pair
__global__ void __launch_bounds__(1024) moe_group_rows_kernel(const MoeRoute a) {
  __shared__ int cnt[kMaxExperts], row0[kMaxExperts], tile0[kMaxExperts];
  const uint32_t tid = threadIdx.x, pairs = a.M * a.top;
  cnt[tid] = 0;
  __syncthreads();
  constexpr uint32_t U = 8;   // pairs a thread has in flight
  for (uint32_t p0 = tid; p0 < pairs; p0 += U * 1024) {
    int e[U];
#pragma unroll
    for (uint32_t u = 0; u < U; u++) e[u] = a.sel[p0 + u * 1024 < pairs ? p0 + u * 1024 : p0];
#pragma unroll
    for (uint32_t u = 0; u < U; u++)
      if (p0 + u * 1024 < pairs && (uint32_t)e[u] < a.experts) atomicAdd(&cnt[e[u]], 1);
  }
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
  for (uint32_t p0 = tid; p0 < pairs; p0 += U * 1024) {
    int e[U];
    float w[U];
#pragma unroll
    for (uint32_t u = 0; u < U; u++) {
      const uint32_t p = p0 + u * 1024 < pairs ? p0 + u * 1024 : p0;
      e[u] = a.sel[p];
      w[u] = a.w[p];
    }
#pragma unroll
    for (uint32_t u = 0; u < U; u++) {
      const uint32_t p = p0 + u * 1024;
      if (p >= pairs) break;
      if ((uint32_t)e[u] >= a.experts) { a.slot[p] = -1; continue; }   // identity: no row
      const int r = atomicAdd(&cnt[e[u]], 1);
      a.slot[p] = r;
      a.src[r] = (int)(p / a.top);
      a.roww[r] = w[u];
    }
  }
}

uint32_t moe_max_tiles(uint32_t rows, uint32_t experts, uint32_t bm) { return rows / bm + (rows < experts ? rows : experts); }

hipError_t moe_route_launch(const MoeRoute& a, bool f32, hipStream_t st) {
  static_assert(kMaxExperts == 1024, "one thread per expert");
  static bool o32[64] = {}, o16[64] = {};
  if (!a.x || !a.router || a.kp % 64 || a.ldx < a.kp || a.M == 0 || a.top == 0 || a.top > a.experts + a.route.identity || a.top > kMaxTop || a.experts > kMaxExperts || a.bm == 0 || a.tiles < moe_max_tiles(a.M * a.top, a.experts, a.bm))
    return hipErrorInvalidValue;
  const uint32_t ne = a.experts + a.route.identity, ep = (ne + 3) & ~3u;
  const bool grp = a.route.form == LGH_ROUTER_SOFTMAX_GROUPS;
  if (grp ? !route_ok(a.route, ne, a.top) : a.route.form != LGH_ROUTER_SIGMOID || a.route.identity) return hipErrorInvalidValue;
  const size_t lds = (size_t)kRouteTokens * (grp ? 2 * ep + a.route.groups + 2 * a.top : ep) * 4;
  const dim3 grid((a.M + kRouteTokens - 1) / kRouteTokens);
  if (ne <= 16) {
    if (f32) hipLaunchKernelGGL((moe_topk_kernel<float, 1>), grid, dim3(512), lds, st, a);
    else hipLaunchKernelGGL((moe_topk_kernel<__bf16, 1>), grid, dim3(512), lds, st, a);
  } else if (f32) {
    if (hipError_t e = lds_opt_in(reinterpret_cast<const void*>(&moe_topk_kernel<float, 4>), 112 * 1024, o32); e != hipSuccess) return e;
    hipLaunchKernelGGL((moe_topk_kernel<float, 4>), grid, dim3(512), lds, st, a);
  } else {
    if (hipError_t e = lds_opt_in(reinterpret_cast<const void*>(&moe_topk_kernel<__bf16, 4>), 112 * 1024, o16); e != hipSuccess) return e;
    hipLaunchKernelGGL((moe_topk_kernel<__bf16, 4>), grid, dim3(512), lds, st, a);
  }
  hipLaunchKernelGGL(moe_group_rows_kernel, dim3(1), dim3(1024), 0, st, a);
  return hipGetLastError();
}

}  // namespace lgh
