// linear_bf16.hip — matrix products with weights kept in bf16 (layered.h): the decode mat-vec (weights streamed once, input vector
// prepared in LDS by every workgroup: residual + layer norm, matrix-memory read-out) and the block product on the matrix cores.
#include "layered.h"
#include "layered_device.h"

namespace lgh {

// ------------------------------------------------------------------------------------------------
// decode mat-vec: one workgroup of 16 waves per CU, so that preparing the input vector (layer norm, read-out) costs a CU once.  A team
// of `ks` waves takes 4 rows at a time and shares their columns; every lane keeps two passes of 4 rows x 16 bytes in flight, across row
// groups, and the first of them are requested before the input vector is prepared.
// ------------------------------------------------------------------------------------------------
constexpr int kMvR = 4;
constexpr uint32_t kMvThreads = 1024;

// layer norm of the K values in xs (in place), times w
__device__ __forceinline__ void ln_lds(float* xs, uint32_t K, const float* w, float eps, float* red) {
  float s = 0.0f;
  for (uint32_t i = threadIdx.x; i < K; i += kMvThreads) s += xs[i];
  const float mean = block_sum(s, red) / (float)K;
  float v = 0.0f;
  for (uint32_t i = threadIdx.x; i < K; i += kMvThreads) { const float d = xs[i] - mean; v = __builtin_fmaf(d, d, v); }
  const float inv = 1.0f / __builtin_sqrtf(block_sum(v, red) / (float)K + eps);
  for (uint32_t i = threadIdx.x; i < K; i += kMvThreads) xs[i] = (xs[i] - mean) * inv * w[i];
}

// row r of group g: 4 consecutive rows, or 2 pairs (a gate row and the up row 16 below it)
__device__ __forceinline__ uint32_t mv_row_of(uint32_t paired, uint32_t g, int r) {
  if (paired) { const uint32_t p = g * 2 + (r & 1); return (p >> 4) * 32 + (p & 15) + (r >> 1) * 16; }
  return g * kMvR + r;
}
__device__ __forceinline__ const uint16_t* mv_row(const LinMv& a, uint32_t g, int r) {
  const uint32_t row = mv_row_of(a.paired, g, r);
  return a.w + (size_t)(row < a.n ? row : a.n - 1) * a.kp;
}
struct MvW { u32x4 w[kMvR]; };
// lanes past the row's end re-read its first bytes (unconditional loads) and add nothing.  g1: groups of the first matrix (LS_TWO) or of
// one expert (LS_EXPERTS); sel: the chosen experts, in LDS
template <int SRC>
__device__ __forceinline__ void mv_fetch(const LinMv& a, uint32_t g, uint32_t kb, uint32_t g1, const int* sel, MvW& o) {
  const uint32_t kc = kb < a.kp ? kb : 0;
  if (SRC == LS_TWO && g >= g1) {
#pragma unroll
    for (int r = 0; r < kMvR; r++) {
      const uint32_t row = (g - g1) * kMvR + r;
      o.w[r] = ldg_nt128(a.w2 + (size_t)(row < a.n2 ? row : a.n2 - 1) * a.kp + kc);
    }
  } else if (SRC == LS_EXPERTS) {
    const uint32_t slot = g / g1, gl = g - slot * g1, ex = (uint32_t)__builtin_amdgcn_readfirstlane(sel[slot]);
    if (ex >= a.experts) {   // (an identity expert has no rows)
#pragma unroll
      for (int r = 0; r < kMvR; r++) o.w[r] = (u32x4)(0u);
      return;
    }
    const uint16_t* w = a.w2 + (size_t)ex * a.stride + kc;
#pragma unroll
    for (int r = 0; r < kMvR; r++) {
      const uint32_t row = mv_row_of(1, gl, r);
      o.w[r] = ldg_nt128(w + (size_t)(row < a.n ? row : a.n - 1) * a.kp);
    }
  } else if (SRC == LS_MOE_DOWN) {
    const uint16_t* w = a.w + kc;
    uint32_t ld = a.kps;
    if (kc >= a.kps) {
      const uint32_t q = kc - a.kps, s = q / a.kpe;
      if ((uint32_t)sel[s] >= a.experts) {
#pragma unroll
        for (int r = 0; r < kMvR; r++) o.w[r] = (u32x4)(0u);
        return;
      }
      w = a.w2 + (size_t)sel[s] * a.stride + (q - s * a.kpe);
      ld = a.kpe;
    }
#pragma unroll
    for (int r = 0; r < kMvR; r++) {
      const uint32_t row = g * kMvR + r;
      o.w[r] = ldg_nt128(w + (size_t)(row < a.n ? row : a.n - 1) * ld);
    }
  } else {
#pragma unroll
    for (int r = 0; r < kMvR; r++) o.w[r] = ldg_nt128(mv_row(a, g, r) + kc);
  }
}
__device__ __forceinline__ void mv_acc(const MvW& o, f32x4 x0, f32x4 x1, float* acc) {
#pragma unroll
  for (int r = 0; r < kMvR; r++) {
    const u32x4 w = o.w[r];
    float s = acc[r];
    s = __builtin_fmaf(bf_lo(w.x), x0.x, s); s = __builtin_fmaf(bf_hi(w.x), x0.y, s);
    s = __builtin_fmaf(bf_lo(w.y), x0.z, s); s = __builtin_fmaf(bf_hi(w.y), x0.w, s);
    s = __builtin_fmaf(bf_lo(w.z), x1.x, s); s = __builtin_fmaf(bf_hi(w.z), x1.y, s);
    s = __builtin_fmaf(bf_lo(w.w), x1.z, s); s = __builtin_fmaf(bf_hi(w.w), x1.w, s);
    acc[r] = s;
  }
}
// what becomes of an unpaired row's sum
__device__ __forceinline__ float mv_row_out(const LinMv& a, float v) {
  if (a.act == LA_RELU2) { const float r = fmaxf(v, 0.0f); return r * r; }
  return a.cap > 0.0f ? a.cap * tanh_f(v / a.cap) : v;
}
// sum over the workgroup, one barrier; red: 16 floats of LDS that nothing else uses
__device__ __forceinline__ float mv_block_sum(float v, float* red) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  f32x4 t = *reinterpret_cast<const f32x4*>(red);
#pragma unroll
  for (int i = 4; i < 16; i += 4) t += *reinterpret_cast<const f32x4*>(red + i);
  return (t.x + t.y) + (t.z + t.w);
}
__device__ __forceinline__ float mv_glu(const LinMv& a, float gate, float up) {
  if (a.act == LA_CLAMPED) return clamped_glu_f(gate, up, a.limit);
  return (a.act == LA_SILU ? silu_f(gate) : gelu_tanh_f(gate)) * up;
}

// mean and 1 / sqrt(variance + eps) of the workgroup's K values, U per thread (channel tid + u * kMvThreads), with one barrier: every wave takes its own
// mean and squared deviations, which are then put together.  st: [3][16] floats of LDS that nothing else uses
template <int U> __device__ __forceinline__ void mv_layer_stats(const float* v, uint32_t K, float eps, float (*st)[16], float& mean, float& inv) {
  const uint32_t wave = threadIdx.x >> 6;
  float n = 0.0f, s = 0.0f, q = 0.0f;
#pragma unroll
  for (int u = 0; u < U; u++) {
    const uint32_t c0 = wave * 64 + u * kMvThreads;
    n += (float)(c0 < K ? (K - c0 < 64 ? K - c0 : 64u) : 0u);
    s += threadIdx.x + u * kMvThreads < K ? v[u] : 0.0f;
  }
  const float mw = wave_total(s) / fmaxf(n, 1.0f);
#pragma unroll
  for (int u = 0; u < U; u++) { const float d = v[u] - mw; q = threadIdx.x + u * kMvThreads < K ? __builtin_fmaf(d, d, q) : q; }
  q = wave_total(q);
  if ((threadIdx.x & 63) == 0) { st[0][wave] = n; st[1][wave] = mw; st[2][wave] = q; }
  __syncthreads();
  f32x4 nn[4], mm[4], t = (f32x4)(0.0f);
#pragma unroll
  for (int i = 0; i < 4; i++) {
    nn[i] = *reinterpret_cast<const f32x4*>(&st[0][i * 4]);
    mm[i] = *reinterpret_cast<const f32x4*>(&st[1][i * 4]);
    t += nn[i] * mm[i];
  }
  const float rk = 1.0f / (float)K;
  mean = ((t.x + t.y) + (t.z + t.w)) * rk;
  t = (f32x4)(0.0f);
#pragma unroll
  for (int i = 0; i < 4; i++) { const f32x4 d = mm[i] - mean; t += *reinterpret_cast<const f32x4*>(&st[2][i * 4]) + nn[i] * d * d; }
  inv = 1.0f / __builtin_sqrtf(((t.x + t.y) + (t.z + t.w)) * rk + eps);
}

// PRO: LinPro; LP_SANDWICH + 256 U: up to U values per thread, in registers
template <int PRO, int SRC, bool POST>
__global__ void __launch_bounds__(kMvThreads) lin_mv_kernel(const LinMv a, uint32_t n_groups, uint32_t ks, uint32_t g1) {
  constexpr bool MOE = SRC == LS_EXPERTS || SRC == LS_MOE_DOWN;
  extern __shared__ __attribute__((aligned(16))) float xs[];   // [kp]
  __shared__ float red[2][16][kMvR];
  __shared__ __attribute__((aligned(16))) float bred[PRO == LP_SANDWICH ? 64 : 16];
  __shared__ __attribute__((aligned(16))) float lst[PRO > 255 ? 2 : 1][3][16];
  __shared__ __attribute__((aligned(16))) float zs[SRC == LS_EXPERTS ? kMaxExperts : 4];
  __shared__ __attribute__((aligned(16))) float zc[SRC == LS_EXPERTS ? 2 * kMaxRouted : 4];   // choice scores, groups
  __shared__ float id_w;
  __shared__ int sel[MOE ? kMaxTop : 1];
  __shared__ float selw[SRC == LS_EXPERTS ? kMaxTop : 1];
  const uint32_t tid = threadIdx.x, lane = tid & 63, wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6));
  const uint32_t team = wave / ks, sub = wave % ks, teams = 16 / ks;
  const uint32_t kb0 = (sub * 64 + lane) * 8, kstep = ks * 512, passes = (a.kp + kstep - 1) / kstep;
  const uint32_t gstep = gridDim.x * teams;
  uint32_t g = blockIdx.x + gridDim.x * team;
  uint32_t gf = g, pf = 0;   // the next pass to request
  MvW n0, n1;
  auto request = [&](MvW& o) {
    if (gf < n_groups) mv_fetch<SRC>(a, gf, kb0 + pf * kstep, g1, sel, o);
    if (++pf == passes) { pf = 0; gf += gstep; }
  };
  if (!MOE) { request(n0); request(n1); }
  int pos = 0;
  float palpha = 0.0f, nalpha = 0.0f;
  if (POST) { pos = __builtin_amdgcn_readfirstlane(*a.post.pos); palpha = *a.post.post.alpha; nalpha = *a.post.next.alpha; }
  if (SRC == LS_EXPERTS) {
    const uint32_t ne = a.experts + a.route.identity, ep = (ne + 3) & ~3u;
    for (uint32_t e = tid; e < ep; e += kMvThreads) zs[e] = e < ne ? rank_key(a.logits[e]) : -INFINITY;
  }
  if (SRC == LS_MOE_DOWN)
    for (uint32_t e = tid; e < a.top; e += kMvThreads) sel[e] = a.sel[e];
  if (PRO == LP_COPY) {
    for (uint32_t i = tid; i < a.k; i += kMvThreads) xs[i] = a.x[i];
  } else if (PRO == LP_PRE) {
    constexpr uint32_t U = 4;   // channels a thread has in flight, their norm weights with them
    float s = 0.0f, nw[U];
    for (uint32_t i0 = tid; i0 < a.k; i0 += U * kMvThreads) {
      float v[U], y[U];
#pragma unroll
      for (uint32_t u = 0; u < U; u++) {
        const uint32_t i = i0 + u * kMvThreads, ic = i < a.k ? i : a.k - 1;
        v[u] = a.x[ic];
        y[u] = a.y ? a.y[ic] : 0.0f;
        if (i0 == tid) nw[u] = a.nw2[ic];
      }
#pragma unroll
      for (uint32_t u = 0; u < U; u++) {
        const uint32_t i = i0 + u * kMvThreads;
        if (i >= a.k) break;
        const float x = __builtin_fmaf(a.mult, y[u], v[u]);
        xs[i] = x;
        if (a.y && blockIdx.x == 0) a.xout[i] = x;
        s = __builtin_fmaf(x, x, s);
      }
    }
    const float inv = 1.0f / __builtin_sqrtf(block_sum(s, bred) / (float)a.k + a.eps) * a.in_scale;
    for (uint32_t i0 = tid; i0 < a.k; i0 += U * kMvThreads)
#pragma unroll
      for (uint32_t u = 0; u < U; u++) {
        const uint32_t i = i0 + u * kMvThreads;
        if (i >= a.k) break;
        const float h = xs[i] * inv * (a.nw_add + (i0 == tid ? nw[u] : a.nw2[i]));
        xs[i] = h;
        if (a.hout && blockIdx.x == 0) a.hout[i] = h;
      }
  } else if constexpr (PRO > 255) {
    constexpr int U = PRO >> 8;
    float v[U], y[U], w1[U], w2[U], mean, inv;
#pragma unroll
    for (int u = 0; u < U; u++) {
      const uint32_t i = tid + u * kMvThreads, ic = i < a.k ? i : a.k - 1;
      if (a.y) { y[u] = a.y[ic]; if (U <= 4) w1[u] = a.nw[ic]; }
      v[u] = a.x[ic];
      if (U <= 4) w2[u] = a.nw2[ic];   // (more of them do not fit the registers)
    }
    if (a.y) {
      mv_layer_stats<U>(y, a.k, a.eps, lst[0], mean, inv);
#pragma unroll
      for (int u = 0; u < U; u++) {
        const uint32_t i = tid + u * kMvThreads;
        v[u] = __builtin_fmaf(a.mult, (y[u] - mean) * inv * (U <= 4 ? w1[u] : a.nw[i < a.k ? i : a.k - 1]), v[u]);
        if (blockIdx.x == 0 && i < a.k) a.xout[i] = v[u];
      }
    }
    mv_layer_stats<U>(v, a.k, a.eps, lst[1], mean, inv);
#pragma unroll
    for (int u = 0; u < U; u++) {
      const uint32_t i = tid + u * kMvThreads;
      if (i < a.k) xs[i] = (v[u] - mean) * inv * (U <= 4 ? w2[u] : a.nw2[i]);
    }
  } else if (PRO == LP_SANDWICH) {
    constexpr uint32_t U = 4;   // channels a thread has in flight, with everything they need
    float v[U], y[U], w1[U], w2[U];
#pragma unroll
    for (uint32_t u = 0; u < U; u++) {
      const uint32_t i = tid + u * kMvThreads, ic = i < a.k ? i : a.k - 1;
      v[u] = a.x[ic];
      w2[u] = a.nw2[ic];
      if (a.y) { y[u] = a.y[ic]; w1[u] = a.nw[ic]; }
    }
    const float n = 1.0f / (float)a.k;
    auto each = [&](auto f) {   // (thread, channel, its place among the first)
      for (uint32_t i0 = tid; i0 < a.k; i0 += U * kMvThreads)
#pragma unroll
        for (uint32_t u = 0; u < U; u++)
          if (i0 + u * kMvThreads < a.k) f(i0 + u * kMvThreads, u, i0 == tid);
    };
    if (a.y) {
      float s = 0.0f, q = 0.0f;
      each([&](uint32_t i, uint32_t u, bool first) { const float z = first ? y[u] : a.y[i]; xs[i] = z; s += z; });
      const float mean = mv_block_sum(s, bred) * n;
      each([&](uint32_t i, uint32_t, bool) { const float d = xs[i] - mean; q = __builtin_fmaf(d, d, q); });
      const float inv = 1.0f / __builtin_sqrtf(mv_block_sum(q, bred + 16) * n + a.eps);
      each([&](uint32_t i, uint32_t u, bool first) {
        const float z = __builtin_fmaf(a.mult, (xs[i] - mean) * inv * (first ? w1[u] : a.nw[i]), first ? v[u] : a.x[i]);
        xs[i] = z;
        if (blockIdx.x == 0) a.xout[i] = z;
      });
    } else {
      each([&](uint32_t i, uint32_t u, bool first) { xs[i] = first ? v[u] : a.x[i]; });
    }
    float s = 0.0f, q = 0.0f;
    each([&](uint32_t i, uint32_t, bool) { s += xs[i]; });
    const float mean = mv_block_sum(s, bred + 32) * n;
    each([&](uint32_t i, uint32_t, bool) { const float d = xs[i] - mean; q = __builtin_fmaf(d, d, q); });
    const float inv = 1.0f / __builtin_sqrtf(mv_block_sum(q, bred + 48) * n + a.eps);
    each([&](uint32_t i, uint32_t u, bool first) { xs[i] = (xs[i] - mean) * inv * (first ? w2[u] : a.nw2[i]); });
  } else if (PRO == LP_READ) {
    for (uint32_t h = wave; h < a.heads; h += 16) {
      const float* num = a.num + (size_t)h * a.ldo;
      const float* gt = a.gate + h * a.vdim;
      float v[4], w[4], z[4], ss = 0.0f;
#pragma unroll
      for (int j = 0; j < 4; j++) {   // everything a lane needs of the first 256 values requested at once
        const uint32_t e = lane + j * 64, ec = e < a.vdim ? e : 0;
        v[j] = num[ec]; w[j] = a.nw[ec]; z[j] = gt[ec];
        ss = __builtin_fmaf(e < a.vdim ? v[j] : 0.0f, v[j], ss);
      }
      for (uint32_t e = lane + 256; e < a.vdim; e += 64) ss = __builtin_fmaf(num[e], num[e], ss);
      const float r = 1.0f / __builtin_sqrtf(wave_total(ss) / (float)a.vdim + a.eps);
#pragma unroll
      for (int j = 0; j < 4; j++) {
        const uint32_t e = lane + j * 64;
        if (e < a.vdim) xs[h * a.vdim + e] = v[j] * r * w[j] * silu_f(z[j]);
      }
      for (uint32_t e = lane + 256; e < a.vdim; e += 64) xs[h * a.vdim + e] = num[e] * r * a.nw[e] * silu_f(gt[e]);
    }
  } else if (PRO == LP_RESID || PRO == LP_HEAD) {
    for (uint32_t i = tid; i < a.k; i += kMvThreads) xs[i] = a.y[i];
    ln_lds(xs, a.k, a.nw, a.eps, bred);
    for (uint32_t i = tid; i < a.k; i += kMvThreads) {
      const float v = a.x[i] + a.mult * xs[i];
      xs[i] = v;
      if (blockIdx.x == 0) a.xout[i] = v;
    }
    if (PRO == LP_HEAD) ln_lds(xs, a.k, a.nw2, a.eps, bred);
  } else {
    for (uint32_t h = wave; h < a.heads; h += 16) {
      const float* num = a.num + (size_t)h * a.ldo;
      const float* nw = a.nw + h * a.vdim;
      const float* gt = a.gate + h * a.vdim;
      const float den = num[a.vdim], em = num[a.vdim + 1];
      if (a.vdim <= 512) {   // everything a lane needs of the head requested at once
        float v[8], w[8], z[8];
#pragma unroll
        for (int j = 0; j < 8; j++) {
          const uint32_t e = lane + j * 64, ec = e < a.vdim ? e : 0;
          v[j] = num[ec]; w[j] = nw[ec]; z[j] = gt[ec];
          if (e >= a.vdim) v[j] = 0.0f;
        }
        const float inv = 1.0f / (fmaxf(fabsf(den), em) + 1e-6f);
        float ss = 0.0f;
#pragma unroll
        for (int j = 0; j < 8; j++) { v[j] *= inv; ss = __builtin_fmaf(v[j], v[j], ss); }
        const float r = 1.0f / __builtin_sqrtf(wave_sum(ss) / (float)a.vdim + a.eps);
#pragma unroll
        for (int j = 0; j < 8; j++) {
          const uint32_t e = lane + j * 64;
          if (e < a.vdim) xs[h * a.vdim + e] = v[j] * r * w[j] * sigmoid_f(z[j]);
        }
      } else {
        const float inv = 1.0f / (fmaxf(fabsf(den), em) + 1e-6f);
        float ss = 0.0f;
        for (uint32_t j = lane; j < a.vdim; j += 64) { const float o = num[j] * inv; ss = __builtin_fmaf(o, o, ss); }
        const float r = 1.0f / __builtin_sqrtf(wave_sum(ss) / (float)a.vdim + a.eps);
        for (uint32_t j = lane; j < a.vdim; j += 64) xs[h * a.vdim + j] = num[j] * inv * r * nw[j] * sigmoid_f(gt[j]);
      }
    }
  }
  for (uint32_t i = a.k + tid; i < a.kp; i += kMvThreads) xs[i] = 0.0f;
  __syncthreads();
  if (SRC == LS_EXPERTS) {
    if (a.route.form == LGH_ROUTER_SIGMOID) {
      for (uint32_t e = tid; e < a.experts; e += kMvThreads) rank_expert(zs, a.experts, a.top, e, sel, selw);
      __syncthreads();
    } else {
      const uint32_t ne = a.experts + a.route.identity;
      route_groups(zs, zc, zc + kMaxRouted, 1, ne, (ne + 3) & ~3u, a.top, a.route, sel, selw);
    }
    if (blockIdx.x == 0 && tid < a.top) {
      a.sel[tid] = sel[tid];
      if (a.selw) a.selw[tid] = selw[tid];
    }
  }
  if (SRC == LS_MOE_DOWN) {
    if (tid == 0) {
      float s = 0.0f;
      if (a.id_x)
        for (uint32_t t = 0; t < a.top; t++) s += (uint32_t)sel[t] >= a.experts ? a.selw[t] : 0.0f;
      id_w = s;
    }
    __syncthreads();
  }
  if (MOE) { request(n0); request(n1); }
  const uint32_t rounds = (n_groups + gstep - 1) / gstep;   // the same for every wave: the teams meet at a barrier when ks > 1
  for (uint32_t rd = 0; rd < rounds; rd++, g += gstep) {
    float acc[kMvR] = {0.0f, 0.0f, 0.0f, 0.0f};
    const uint32_t ch = g * kMvR + (lane & 3);   // POST: the channel this lane finishes
    PostIn pi;
    if (POST && sub == 0) post_fetch(a.post, ch < a.n ? ch : a.n - 1, pos, pi);
    if (g < n_groups) {
      for (uint32_t p = 0; p < passes; p++) {
        const MvW cur = n0;
        n0 = n1;
        request(n1);
        const uint32_t kb = kb0 + p * kstep;
        if (kb < a.kp) mv_acc(cur, *reinterpret_cast<const f32x4*>(xs + kb), *reinterpret_cast<const f32x4*>(xs + kb + 4), acc);
      }
#pragma unroll
      for (int r = 0; r < kMvR; r++) acc[r] = wave_sum_to_lane63(acc[r]);
    }
    if (ks > 1) {
      if (lane == 63) {
#pragma unroll
        for (int r = 0; r < kMvR; r++) red[rd & 1][wave][r] = acc[r];
      }
      __syncthreads();
      if (sub == 0 && lane == 63) {
#pragma unroll
        for (int r = 0; r < kMvR; r++)
          for (uint32_t k = 1; k < ks; k++) acc[r] += red[rd & 1][wave + k][r];
      }
    }
    if constexpr (POST) {
      if (sub == 0 && g < n_groups) {
        float y[kMvR];
#pragma unroll
        for (int r = 0; r < kMvR; r++) y[r] = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, acc[r]), 63));
        const float v = (lane & 2) ? ((lane & 1) ? y[3] : y[2]) : ((lane & 1) ? y[1] : y[0]);
        if (lane < kMvR && ch < a.n) post_finish(a.post, pi, ch, pos, v, palpha, nalpha);
      }
    } else if (SRC == LS_EXPERTS) {
      if (sub == 0 && lane == 63 && g < n_groups) {
        const uint32_t slot = g / g1, gl = g - slot * g1;
        const float win = a.route.form == LGH_ROUTER_SIGMOID ? selw[slot] : 1.0f, wout = a.route.form == LGH_ROUTER_SIGMOID ? 1.0f : selw[slot];
#pragma unroll
        for (int r = 0; r < 2; r++)
          if (gl * 2 + r < a.n / 2) a.out[(size_t)slot * a.kpe + gl * 2 + r] = wout * mv_glu(a, win * acc[r], win * acc[r + 2]);
      }
    } else if (SRC == LS_TWO && g >= g1) {
      if (sub == 0 && lane == 63 && g < n_groups) {
#pragma unroll
        for (int r = 0; r < kMvR; r++)
          if ((g - g1) * kMvR + r < a.n2) a.out2[(g - g1) * kMvR + r] = acc[r];
      }
    } else if (sub == 0 && lane == 63 && g < n_groups) {
      if (!a.paired) {
#pragma unroll
        for (int r = 0; r < kMvR; r++)
          if (g * kMvR + r < a.n) {
            const uint32_t n = g * kMvR + r;
            float v = acc[r];
            if (a.bias) v += a.bias[n];
            if (SRC == LS_MOE_DOWN && a.id_x) v = __builtin_fmaf(id_w, a.id_x[n], v);
            a.out[n] = SRC == LS_PLAIN ? mv_row_out(a, v) : v;
          }
      } else {
#pragma unroll
        for (int r = 0; r < 2; r++)
          if (g * 2 + r < a.n / 2) a.out[g * 2 + r] = mv_glu(a, acc[r], acc[r + 2]);
      }
    }
  }
}

template <int PRO, int SRC, bool POST>
static hipError_t lin_mv_run(const LinMv& a, hipStream_t st) {
  static bool opted[64] = {};
  if (hipError_t e = lds_opt_in(reinterpret_cast<const void*>(&lin_mv_kernel<PRO, SRC, POST>), (SRC == LS_EXPERTS ? 140 : 152) * 1024, opted); e != hipSuccess) return e;
  const uint32_t g1 = (a.n + kMvR - 1) / kMvR;
  const uint32_t groups = SRC == LS_TWO ? g1 + (a.n2 + kMvR - 1) / kMvR : SRC == LS_EXPERTS ? g1 * a.top : g1;
  uint32_t ks = 1;   // waves per team: enough teams for the groups of a CU, and at least a full pass of columns per wave
  while (ks < 8 && (uint64_t)groups * ks * 2 <= kNumCU * 16 && a.kp >= 1024 * ks) ks *= 2;
  hipLaunchKernelGGL((lin_mv_kernel<PRO, SRC, POST>), dim3(groups < kNumCU ? groups : kNumCU), dim3(kMvThreads), (size_t)a.kp * 4, st, a, groups, ks, g1);
  return hipGetLastError();
}
template <int PRO, int SRC>
static hipError_t lin_mv_post(const LinMv& a, hipStream_t st) {
  if (!a.post.xout) return lin_mv_run<PRO, SRC, false>(a, st);
  const PostUpdate& p = a.post;
  if (a.paired || p.width != a.n || !p.x || !p.hout || !p.pos || !p.post.w || !p.post.b || !p.post.alpha || !p.next.w || !p.next.b || !p.next.alpha ||
      (p.conv.taps && !p.conv.w) || (p.conv.taps > 1 && !p.conv.hist))
    return hipErrorInvalidValue;
  return lin_mv_run<PRO, SRC, true>(a, st);
}
template <int PRO>
static hipError_t lin_mv_go(const LinMv& a, int src, hipStream_t st) {
  if (src == LS_TWO) return a.post.xout || !a.w2 || !a.out2 || a.n2 == 0 ? hipErrorInvalidValue : lin_mv_run<PRO, LS_TWO, false>(a, st);
  return src != LS_PLAIN || a.post.xout ? hipErrorInvalidValue : lin_mv_run<PRO, LS_PLAIN, false>(a, st);
}

bool route_ok(const RouteForm& f, uint32_t outputs, uint32_t top) {
  return f.form == LGH_ROUTER_SOFTMAX_GROUPS && f.correction && outputs <= kMaxRouted && f.groups && outputs % f.groups == 0 && f.keep && f.keep <= f.groups &&
         top && (uint64_t)f.keep * (outputs / f.groups) >= top && f.identity < outputs;
}

hipError_t lin_mv_launch(int pro, const LinMv& a, hipStream_t st, int src) {
  if ((a.bias && (a.paired || a.post.xout)) || ((a.act == LA_RELU2 || a.cap > 0.0f) && (a.paired || a.post.xout || src != LS_PLAIN))) return hipErrorInvalidValue;
  if ((a.n && src != LS_EXPERTS && !a.w && !(src == LS_MOE_DOWN && a.kps == 0)) || (a.n && !a.out && !a.post.xout) || (a.n == 0 && src != LS_TWO) || a.kp % 64 ||
      a.kp > kLinMvMaxK || a.k > a.kp || (a.paired && a.n % 32))
    return hipErrorInvalidValue;
  if (src == LS_EXPERTS || src == LS_MOE_DOWN) {
    if (pro != LP_COPY || !a.x || !a.w2 || !a.sel || a.top == 0 || a.top > kMaxTop || a.kpe % 64) return hipErrorInvalidValue;
    if (src == LS_EXPERTS) {
      const uint32_t ne = a.experts + a.route.identity;
      if (!a.paired || !a.logits || !a.out || ne > kMaxExperts || a.top > ne || a.kpe < a.n / 2) return hipErrorInvalidValue;
      if (a.route.form == LGH_ROUTER_SIGMOID ? a.route.identity != 0 : !route_ok(a.route, ne, a.top) || !a.selw) return hipErrorInvalidValue;
      return lin_mv_run<LP_COPY, LS_EXPERTS, false>(a, st);
    }
    if (a.paired || a.kps % 64 || a.kpe == 0 || a.kp != a.kps + a.top * a.kpe || !a.experts || (a.id_x && (!a.selw || a.post.xout))) return hipErrorInvalidValue;
    return lin_mv_post<LP_COPY, LS_MOE_DOWN>(a, st);
  }
  switch (pro) {
    case LP_COPY:
      if (!a.x) return hipErrorInvalidValue;
      return src == LS_PLAIN ? lin_mv_post<LP_COPY, LS_PLAIN>(a, st) : lin_mv_go<LP_COPY>(a, src, st);
    case LP_RESID: return a.x && a.y && a.nw && a.xout ? lin_mv_go<LP_RESID>(a, src, st) : hipErrorInvalidValue;
    case LP_HEAD: return a.x && a.y && a.nw && a.nw2 && a.xout && src == LS_PLAIN && !a.post.xout ? lin_mv_run<LP_HEAD, LS_PLAIN, false>(a, st) : hipErrorInvalidValue;
    case LP_PRE: return a.x && a.nw2 && (!a.y || a.xout) ? lin_mv_go<LP_PRE>(a, src, st) : hipErrorInvalidValue;
    case LP_SANDWICH:
      if (!a.x || !a.nw2 || (a.y && (!a.nw || !a.xout)) || src != LS_PLAIN || a.post.xout) return hipErrorInvalidValue;
      if (a.k <= 1 * kMvThreads) return lin_mv_run<LP_SANDWICH + 256 * 1, LS_PLAIN, false>(a, st);
      if (a.k <= 2 * kMvThreads) return lin_mv_run<LP_SANDWICH + 256 * 2, LS_PLAIN, false>(a, st);
      if (a.k <= 4 * kMvThreads) return lin_mv_run<LP_SANDWICH + 256 * 4, LS_PLAIN, false>(a, st);
      if (a.k <= 8 * kMvThreads) return lin_mv_run<LP_SANDWICH + 256 * 8, LS_PLAIN, false>(a, st);
      return lin_mv_run<LP_SANDWICH, LS_PLAIN, false>(a, st);
    case LP_READ:
      return a.num && a.nw && a.gate && a.heads * a.vdim == a.k && src == LS_PLAIN && !a.post.xout ? lin_mv_run<LP_READ, LS_PLAIN, false>(a, st) : hipErrorInvalidValue;
    case LP_MLSTM:
      return a.num && a.nw && a.gate && a.heads * a.vdim == a.k && src == LS_PLAIN ? lin_mv_post<LP_MLSTM, LS_PLAIN>(a, st) : hipErrorInvalidValue;
  }
  return hipErrorInvalidValue;
}

// ------------------------------------------------------------------------------------------------
// block product.  A workgroup of 4 waves computes BN weight rows x BM tokens, k in steps of 64; both operands go global -> LDS by
// DMA (two buffers), 16-byte chunks of a row stored at chunk ^ (row & mask) so that the 16 rows of a fragment read different banks.
// The weights are the A operand: a lane ends up with 4 consecutive output columns of one token.
// ------------------------------------------------------------------------------------------------
template <class T> constexpr uint32_t act_chunks() { return 64 * sizeof(T) / 16; }   // 16-byte chunks of a row's 64 columns

template <class T, int BM, int BN, int WN, int EPI, bool GRP>
__global__ void __launch_bounds__(256) lin_gemm_kernel(const LinGemm a, uint32_t tiles_n, uint32_t tiles_m) {
  constexpr int WM = 4 / WN, NT = BN / WN / 16, MT = BM / WM / 16;
  constexpr uint32_t XC = act_chunks<T>();
  constexpr uint32_t kWBytes = BN * 128, kXBytes = BM * XC * 16, kBuf = kWBytes + kXBytes;
  extern __shared__ __attribute__((aligned(16))) uint8_t smem[];
  const uint32_t lane = threadIdx.x & 63, wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6));
  // consecutive tiles of one weight panel on one XCD (workgroups go round-robin over the 8 XCDs)
  uint32_t t = blockIdx.x;
  const uint32_t total = tiles_n * tiles_m;
  {
    const uint32_t q = total / 8, r = total % 8, xcd = t % 8, i = t / 8;
    t = xcd * q + (xcd < r ? xcd : r) + i;
  }
  const uint32_t tn = t / tiles_m, tm = t % tiles_m;
  const uint32_t n0 = tn * BN;
  uint32_t m0 = tm * BM, m_end = a.M;   // rows of this tile
  const uint16_t* W = a.w;
  if constexpr (GRP) {
    const int e = a.grp.tile_e[tm];
    if (e < 0) return;
    m0 = (uint32_t)a.grp.tile_row[tm];
    m_end = (uint32_t)a.grp.seg[e + 1];
    W += (size_t)e * a.grp.stride;
  }
  const uint32_t wn = wave % WN, wm = wave / WN;
  const uint32_t r16 = lane & 15, g = lane >> 4;
  const T* X = reinterpret_cast<const T*>(a.x);

  constexpr uint32_t RPI = 64 / XC;                          // rows of x per wave instruction
  constexpr int NX = (int)((kXBytes / 1024 + 3) / 4);
  uint32_t xrow[GRP ? NX : 1];                               // grouped: where this lane's rows lie
  if constexpr (GRP) {
#pragma unroll
    for (int i = 0; i < NX; i++) {
      const uint32_t r = m0 + (i * 4 + wave) * RPI + lane / XC, m = r < m_end ? r : m_end - 1;
      xrow[i] = a.grp.src ? (uint32_t)a.grp.src[m] : m;
    }
  }
  auto stage = [&](uint32_t k0, uint32_t buf) {
    uint8_t* base = smem + buf * kBuf;
#pragma unroll
    for (int i = 0; i < (int)(kWBytes / 4096); i++) {       // weights: 8 chunks a row, a wave instruction covers 8 rows
      const uint32_t row = (i * 4 + wave) * 8 + (lane >> 3), ch = (lane & 7) ^ (row & 7);
      const uint32_t n = n0 + row < a.np ? n0 + row : a.np - 1;
      lds_dma16(W + (size_t)n * a.kp + k0 + ch * 8, base + (i * 4 + wave) * 1024);
    }
#pragma unroll
    for (int i = 0; i < NX; i++) {
      const uint32_t blk = i * 4 + wave;
      if (kXBytes / 1024 % 4 == 0 || blk < kXBytes / 1024) {
        const uint32_t row = blk * RPI + lane / XC, ch = (lane % XC) ^ (row & (XC - 1));
        const uint32_t m = GRP ? xrow[GRP ? i : 0] : m0 + row < a.M ? m0 + row : a.M - 1;
        lds_dma16(X + (size_t)m * a.ldx + k0 + ch * (16 / sizeof(T)), base + kWBytes + blk * 1024);
      }
    }
  };

  f32x4 acc[NT][MT];
#pragma unroll
  for (int i = 0; i < NT; i++)
#pragma unroll
    for (int j = 0; j < MT; j++) acc[i][j] = (f32x4)(0.0f);

  stage(0, 0);
  __builtin_amdgcn_s_waitcnt(0x0F70);   // vmcnt(0)
  __syncthreads();
  const uint32_t steps = a.kp / 64;
  for (uint32_t s = 0; s < steps; s++) {
    const uint32_t cur = s & 1;
    if (s + 1 < steps) stage((s + 1) * 64, cur ^ 1);
    const uint8_t* wb = smem + cur * kBuf;
    const uint8_t* xb = wb + kWBytes;
    constexpr int U = 64 / Frag<T>::KU;
#pragma unroll
    for (int u = 0; u < U; u++) {
      typename Frag<T>::V wf[NT], xf[MT];
#pragma unroll
      for (int i = 0; i < NT; i++) {
        const uint32_t row = (wn * NT + i) * 16 + r16;
        if constexpr (sizeof(T) == 2) {
          wf[i] = *reinterpret_cast<const bf16x8*>(wb + row * 128 + (((uint32_t)(u * 4) + g) ^ (row & 7)) * 16);
        } else {   // 4 bf16 values of the 16-column unit: half a chunk
          const u32x2 h = *reinterpret_cast<const u32x2*>(wb + row * 128 + (((uint32_t)(u * 2) + (g >> 1)) ^ (row & 7)) * 16 + (g & 1) * 8);
          f32x4 v;
          v.x = bf_lo(h.x); v.y = bf_hi(h.x); v.z = bf_lo(h.y); v.w = bf_hi(h.y);
          wf[i] = v;
        }
      }
#pragma unroll
      for (int j = 0; j < MT; j++) {
        const uint32_t row = (wm * MT + j) * 16 + r16;
        xf[j] = Frag<T>::load(reinterpret_cast<const T*>(xb + row * (XC * 16) + (((uint32_t)(u * 4) + g) ^ (row & (XC - 1))) * 16));
      }
#pragma unroll
      for (int i = 0; i < NT; i++)
#pragma unroll
        for (int j = 0; j < MT; j++) acc[i][j] = Frag<T>::mma(wf[i], xf[j], acc[i][j]);
    }
    __builtin_amdgcn_s_waitcnt(0x0F70);
    __syncthreads();
  }
  // lane: token r16 of a token tile, columns 4g .. 4g + 3 of a weight tile
#pragma unroll
  for (int j = 0; j < MT; j++) {
    const uint32_t m = m0 + (wm * MT + j) * 16 + r16;
    if (m >= m_end) continue;
    if constexpr (EPI == LE_GEGLU || EPI == LE_SWIGLU || EPI == LE_CLAMPED) {
      const float in = GRP ? a.grp.scale[m] : 1.0f;            // factor of the row's input
#pragma unroll
      for (int i = 0; i < NT; i += 2) {
        const uint32_t nb = n0 + (wn * NT + i) * 16;           // gate rows; the up rows follow
        if (nb >= a.n) continue;
        T* o = reinterpret_cast<T*>(a.out) + (size_t)m * a.ldo + nb / 2 + g * 4;
#pragma unroll
        for (int e = 0; e < 4; e++) {
          if constexpr (EPI == LE_CLAMPED) { o[e] = to_act<T>(in * clamped_glu_f(acc[i][j][e], acc[i + 1][j][e], a.grp.limit)); continue; }
          const float gt = GRP ? in * acc[i][j][e] : acc[i][j][e], u = GRP ? in * acc[i + 1][j][e] : acc[i + 1][j][e];
          o[e] = to_act<T>((EPI == LE_SWIGLU ? silu_f(gt) : gelu_tanh_f(gt)) * u);
        }
      }
    } else {
#pragma unroll
      for (int i = 0; i < NT; i++) {
        const uint32_t nb = n0 + (wn * NT + i) * 16 + g * 4;
        if constexpr (EPI == LE_F32) {
          float* o = reinterpret_cast<float*>(a.out) + (size_t)m * a.ldo + nb;
          if (a.bias) {
#pragma unroll
            for (int e = 0; e < 4; e++) acc[i][j][e] += a.bias[nb + e < a.n ? nb + e : a.n - 1];
          }
          if (a.cap > 0.0f) {
#pragma unroll
            for (int e = 0; e < 4; e++) acc[i][j][e] = a.cap * tanh_f(acc[i][j][e] / a.cap);
          }
          if (nb + 4 <= a.n && (a.ldo & 3) == 0) *reinterpret_cast<f32x4*>(o) = acc[i][j];
          else
            for (int e = 0; e < 4; e++)
              if (nb + e < a.n) o[e] = acc[i][j][e];
        } else if constexpr (EPI == LE_RELU2) {
          T* o = reinterpret_cast<T*>(a.out) + (size_t)m * a.ldo + nb;
          T r[4];
#pragma unroll
          for (int e = 0; e < 4; e++) { const float v = fmaxf(acc[i][j][e], 0.0f); r[e] = to_act<T>(v * v); }
          if (nb + 4 <= a.n) __builtin_memcpy(__builtin_assume_aligned(o, sizeof(r)), r, sizeof(r));   // (rows are multiples of 64)
          else
            for (int e = 0; e < 4; e++)
              if (nb + e < a.n) o[e] = r[e];
        } else if constexpr (EPI == LE_ACT) {
          T* o = reinterpret_cast<T*>(a.out) + (size_t)m * a.ldo + nb;
#pragma unroll
          for (int e = 0; e < 4; e++)
            if (nb + e < a.n) o[e] = to_act<T>(acc[i][j][e]);
        } else if (EPI == LE_HEADS && (a.hd & 3) == 0 && nb + 4 <= a.n) {   // the four columns lie in one head
          T* o = reinterpret_cast<T*>(a.out) + ((size_t)(nb / a.hd) * a.tcap + m) * a.ldo + nb % a.hd;
          T v[4];
#pragma unroll
          for (int e = 0; e < 4; e++) v[e] = to_act<T>(acc[i][j][e]);
          __builtin_memcpy(__builtin_assume_aligned(o, sizeof(v)), v, sizeof(v));
        } else {
#pragma unroll
          for (int e = 0; e < 4; e++) {
            const uint32_t n = nb + e;
            if (n >= a.n) break;
            const uint32_t h = n / a.hd, d = n % a.hd;
            const size_t at = EPI == LE_HEADS ? ((size_t)h * a.tcap + m) * a.ldo + d : ((size_t)h * a.hrows + d) * a.ldo + m;
            reinterpret_cast<T*>(a.out)[at] = to_act<T>(acc[i][j][e]);
          }
        }
      }
    }
  }
}

template <class T, int BM, int BN, int WN, int EPI, bool GRP = false>
static hipError_t lin_gemm_go(const LinGemm& a, hipStream_t st) {
  static bool opted[64] = {};
  constexpr size_t lds = 2 * (BN * 128 + (size_t)BM * act_chunks<T>() * 16);
  if (hipError_t e = lds_opt_in(reinterpret_cast<const void*>(&lin_gemm_kernel<T, BM, BN, WN, EPI, GRP>), (int)lds, opted); e != hipSuccess) return e;
  const uint32_t tn = (a.n + BN - 1) / BN, tm = GRP ? a.grp.tiles : (a.M + BM - 1) / BM;
  hipLaunchKernelGGL((lin_gemm_kernel<T, BM, BN, WN, EPI, GRP>), dim3(tn * tm), dim3(256), lds, st, a, tn, tm);
  return hipGetLastError();
}

template <class T, int EPI>
static hipError_t lin_gemm_pick(const LinGemm& a, hipStream_t st) {
  const uint32_t tn = (a.n + 127) / 128;
  if (a.M > 64 && tn * ((a.M + 127) / 128) >= 224) return lin_gemm_go<T, 128, 128, 2, EPI>(a, st);
  if (a.M > 32 && tn * ((a.M + 63) / 64) >= 160) return lin_gemm_go<T, 64, 128, 4, EPI>(a, st);
  if (a.M > 16) return lin_gemm_go<T, 32, 128, 4, EPI>(a, st);
  return lin_gemm_go<T, 16, 128, 4, EPI>(a, st);
}

uint32_t lin_group_rows(uint32_t rows, uint32_t groups) {
  const uint32_t avg = rows / groups;
  return avg > 96 ? 128 : avg > 40 ? 64 : avg > 16 ? 32 : 16;
}
template <class T, int EPI>
static hipError_t lin_gemm_group(const LinGemm& a, hipStream_t st) {
  switch (a.grp.bm) {
    case 128: return lin_gemm_go<T, 128, 128, 2, EPI, true>(a, st);
    case 64: return lin_gemm_go<T, 64, 128, 4, EPI, true>(a, st);
    case 32: return lin_gemm_go<T, 32, 128, 4, EPI, true>(a, st);
    case 16: return lin_gemm_go<T, 16, 128, 4, EPI, true>(a, st);
  }
  return hipErrorInvalidValue;
}

hipError_t lin_gemm_launch(int epi, bool f32, const LinGemm& a, hipStream_t st) {
  const uint32_t el = f32 ? 4 : 2;
  if (!a.w || !a.x || !a.out || a.n == 0 || a.M == 0 || a.kp % 64 || a.ldx < a.kp || (a.ldx * el) % 16 || a.np % 16 || a.n > a.np) return hipErrorInvalidValue;
  if ((epi == LE_RELU2 && a.ldo % 64) || (a.cap > 0.0f && (epi != LE_F32 || a.grp.tiles))) return hipErrorInvalidValue;
  if ((epi == LE_GEGLU || epi == LE_SWIGLU || epi == LE_CLAMPED) && a.n % 32) return hipErrorInvalidValue;
  if (a.grp.tiles) {
    if (!a.grp.seg || !a.grp.tile_e || !a.grp.tile_row || ((epi == LE_SWIGLU || epi == LE_CLAMPED) && !a.grp.scale)) return hipErrorInvalidValue;
    if (epi == LE_SWIGLU) return f32 ? lin_gemm_group<float, LE_SWIGLU>(a, st) : lin_gemm_group<__bf16, LE_SWIGLU>(a, st);
    if (epi == LE_CLAMPED) return f32 ? lin_gemm_group<float, LE_CLAMPED>(a, st) : lin_gemm_group<__bf16, LE_CLAMPED>(a, st);
    if (epi == LE_F32) return f32 ? lin_gemm_group<float, LE_F32>(a, st) : lin_gemm_group<__bf16, LE_F32>(a, st);
    return hipErrorInvalidValue;
  }
  if ((epi == LE_HEADS || epi == LE_HEADS_T) && !a.hd) return hipErrorInvalidValue;
#define LGH_GEMM_CASE(E) \
  case E: return f32 ? lin_gemm_pick<float, E>(a, st) : lin_gemm_pick<__bf16, E>(a, st);
  switch (epi) {
    LGH_GEMM_CASE(LE_F32)
    LGH_GEMM_CASE(LE_ACT)
    LGH_GEMM_CASE(LE_GEGLU)
    LGH_GEMM_CASE(LE_HEADS)
    LGH_GEMM_CASE(LE_HEADS_T)
    LGH_GEMM_CASE(LE_SWIGLU)
    LGH_GEMM_CASE(LE_RELU2)
  }
#undef LGH_GEMM_CASE
  return hipErrorInvalidValue;
}

// ------------------------------------------------------------------------------------------------
// upload-time layouts
// ------------------------------------------------------------------------------------------------
__global__ void __launch_bounds__(256) lin_pack_kernel(const uint16_t* __restrict__ src, uint32_t k, uint16_t* __restrict__ dst, uint32_t kp, uint32_t row0, int mode) {
  const uint32_t r = blockIdx.y;
  const uint32_t row = mode == 0 ? row0 + r : row0 + (r >> 4) * 32 + (r & 15) + (mode == 2 ? 16 : 0);
  for (uint32_t i = blockIdx.x * 256 + threadIdx.x; i < k; i += gridDim.x * 256) dst[(size_t)row * kp + i] = src[(size_t)r * k + i];
}

hipError_t lin_pack_launch(const uint16_t* src, uint32_t rows, uint32_t k, uint16_t* dst, uint32_t kp, uint32_t row0, int mode, hipStream_t st) {
  for (uint32_t r = 0; r < rows; r += 32768) {   // (32768: a multiple of the pair block, below the grid's y limit)
    const uint32_t c = rows - r < 32768 ? rows - r : 32768;
    hipLaunchKernelGGL(lin_pack_kernel, dim3((k + 1023) / 1024, c), dim3(256), 0, st, src + (size_t)r * k, k, dst, kp, row0 + (mode ? 2 * r : r), mode);
  }
  return hipGetLastError();
}

__global__ void __launch_bounds__(256) lin_transpose_heads_kernel(const uint16_t* __restrict__ src, uint32_t dim, uint32_t rank, uint16_t* __restrict__ dst, uint32_t dimp) {
  const uint32_t h = blockIdx.y, r = blockIdx.x;
  for (uint32_t d = threadIdx.x; d < dim; d += 256) dst[((size_t)h * rank + r) * dimp + d] = src[((size_t)h * dim + d) * rank + r];
}

hipError_t lin_transpose_heads_launch(const uint16_t* src, uint32_t heads, uint32_t dim, uint32_t rank, uint16_t* dst, uint32_t dimp, hipStream_t st) {
  hipLaunchKernelGGL(lin_transpose_heads_kernel, dim3(rank, heads), dim3(256), 0, st, src, dim, rank, dst, dimp);
  return hipGetLastError();
}

}  // namespace lgh
