// tied_attention.hip — grouped softmax attention whose values are its keys (layered.h): the value of a position is its key as projected,
// the key is that row divided by the root mean square of ALL the position's key heads, times a norm weight.  So a position is cached once,
// unnormed, beside one factor (kinv); the norm weights of queries and keys, the head's temperature and the scale go into the query.
//
//   score(i, j) = cap * tanh(q_i . k_j * kinv_j / cap) - 2^(-8 (h + 1) / heads) * (i - j),   j <= i and (i - j < window or j < keep)
//
// and the softmax's denominator has one more term, exp(sink_h).  Scores, softmax and sums are in 32-bit, in units of log2.
//
//   decode and short portions: a workgroup = one key head x one share of the visible keys; a lane holds 16 bytes of a few keys' rows in
//     registers, for the score and for the weighted sum; only visible keys are touched (kept ones and the window, counted through).
//   prompt portions: causal flash attention in the transposed form of the latent kernel, the key tile serving as the value tile.
#include <algorithm>

#include "layered.h"
#include "layered_device.h"

namespace lgh {

constexpr float kTiedNeg = -1e30f, kTiedLog2e = 1.4426950408889634f;

// cap * tanh(x / cap) in units of log2, of u = x / cap (cap 0: x itself, of u = x); the queries carry the factor 1 / cap
__device__ __forceinline__ float cap_unit(float cap) { return cap > 0.0f ? 1.0f / cap : 1.0f; }
struct CapF {
  float lim, c0, c1, c2, c3, c4;   // the series of tanh (up to |u| < lim) times cap * log2(e)
  __device__ __forceinline__ explicit CapF(float cap) {
    const float o = cap > 0.0f ? cap * kTiedLog2e : kTiedLog2e, k = cap > 0.0f ? o : 0.0f;
    lim = cap > 0.0f ? 0.25f : INFINITY;
    c0 = o; c1 = k * (-1.0f / 3.0f); c2 = k * (2.0f / 15.0f); c3 = k * (-17.0f / 315.0f); c4 = k * (62.0f / 2835.0f);
  }
  __device__ __forceinline__ float small(float u, float add) const {   // |u| < lim
    const float z = u * u;
    return __builtin_fmaf(u, __builtin_fmaf(z, __builtin_fmaf(z, __builtin_fmaf(z, __builtin_fmaf(z, c4, c3), c2), c1), c0), add);
  }
  __device__ __forceinline__ float small_bf(float u, float add) const {   // to 4e-7 of the score: keys and queries are bf16
    const float z = u * u;
    return __builtin_fmaf(u, __builtin_fmaf(z, __builtin_fmaf(z, __builtin_fmaf(z, c3, c2), c1), c0), add);
  }
  __device__ __forceinline__ float any(float u, float add) const { return fabsf(u) < lim ? small(u, add) : __builtin_fmaf(tanh_f(u), c0, add); }
};
__device__ __forceinline__ float tied_slope(uint32_t h, uint32_t heads) {   // in units of log2
  return exp2f(-8.0f * (float)(h + 1) / (float)heads) * kTiedLog2e;
}

// the keys position i sees, counted through: v < nk are the kept ones, the others lie from lo on
struct TiedSeen { uint32_t lo, nk, total; };
__device__ __host__ __forceinline__ TiedSeen tied_seen(const TiedShape& s, uint32_t i) {
  TiedSeen r;
  r.lo = i + 1 > s.window ? i + 1 - s.window : 0;
  r.nk = s.keep < r.lo ? s.keep : r.lo;
  r.total = r.nk + i + 1 - r.lo;
  return r;
}

// lanes that share a key row in the decode kernel
__host__ __device__ constexpr uint32_t tied_lanes(uint32_t dp, uint32_t el) {
  return dp * el <= 128 ? 8 : dp * el <= 256 ? 16 : dp * el <= 512 ? 32 : 64;
}
constexpr uint32_t kTiedBatch = 4;   // key rows a lane has in flight
__host__ __device__ constexpr uint32_t tied_round(uint32_t lanes) { return 4 * kTiedBatch * (64 / lanes); }   // keys of a workgroup per round

// a thread's share (of 256) of the sum of n squares; its first 16 values requested by `squares_fetch`
struct Squares { f32x4 v[4]; };
__device__ __forceinline__ void squares_fetch(const float* p, uint32_t n, uint32_t i0, Squares& o) {
#pragma unroll
  for (uint32_t u = 0; u < 4; u++) {
    const uint32_t i = i0 + u * 1024;
    if ((n & 3) == 0) { o.v[u] = *reinterpret_cast<const f32x4*>(p + (i < n ? i : 0)); continue; }
#pragma unroll
    for (uint32_t e = 0; e < 4; e++) o.v[u][e] = p[i + e < n ? i + e : 0];
  }
}
__device__ __forceinline__ float squares(const float* p, uint32_t n, Squares in) {
  float s = 0.0f;
  for (uint32_t i0 = threadIdx.x * 4; i0 < n; i0 += 4096) {
    if (i0 >= 4096) squares_fetch(p, n, i0, in);
#pragma unroll
    for (uint32_t u = 0; u < 4; u++)
#pragma unroll
      for (uint32_t e = 0; e < 4; e++) {
        const float x = i0 + u * 1024 + e < n ? in.v[u][e] : 0.0f;
        s = __builtin_fmaf(x, x, s);
      }
  }
  return s;
}

// grid (splits, kv heads * chunks of HQ query heads, tokens)
template <class T, uint32_t LPK, int HQ, bool OWN>
__global__ void __launch_bounds__(256) tied_attn_kernel(const TiedShape s, const TiedBufs b, const int* __restrict__ pos_ptr, uint32_t pos0, uint32_t M, uint32_t n_splits) {
  constexpr int PER = 16 / sizeof(T), NB = kTiedBatch;
  constexpr uint32_t GPW = 64 / LPK, HALF = GPW > 1 ? 32 : 64;      // key groups of a wave; lanes left after folding its halves
  __shared__ float red[16];
  __shared__ float ml[2][4][HQ];
  extern __shared__ __attribute__((aligned(16))) float accs[];      // [4 waves][HQ][HALF][PER]
  const uint32_t tid = threadIdx.x, lane = tid & 63, w = tid >> 6, grp = lane / LPK, sub = lane % LPK;
  const uint32_t gq = s.heads / s.kv_heads, chunks = (gq + HQ - 1) / HQ, g = blockIdx.y / chunks, h0 = g * gq + (blockIdx.y % chunks) * HQ;
  const uint32_t hn = (g + 1) * gq - h0 < (uint32_t)HQ ? (g + 1) * gq - h0 : (uint32_t)HQ, z = blockIdx.z, sp = blockIdx.x;
  const uint32_t pos = (pos_ptr ? (uint32_t)*pos_ptr : pos0) + z;
  const TiedSeen seen = tied_seen(s, pos);
  constexpr uint32_t KR = tied_round(LPK);
  const uint32_t rounds = (seen.total + KR - 1) / KR, per = (rounds + n_splits - 1) / n_splits;
  const uint32_t rb = sp * per, re = rb + per < rounds ? rb + per : rounds;
  if (rb >= re) return;                                             // (the merge skips the same splits)
  const float* cat = b.cat + (size_t)z * s.ldcat;
  T* cache = reinterpret_cast<T*>(b.cache) + (size_t)g * s.rows * s.dp;
  const uint32_t d0 = sub * PER, dc = d0 < s.dp ? d0 : 0;
  u32x4 kraw[NB];
  float kin[NB];
  uint32_t kp[NB];
  auto fetch = [&](uint32_t r) {
#pragma unroll
    for (int i = 0; i < NB; i++) {
      const uint32_t v = (r * 4 + w) * (NB * GPW) + i * GPW + grp, vc = v < seen.total ? v : seen.total - 1;
      const uint32_t p = vc < seen.nk ? vc : seen.lo + vc - seen.nk;
      kp[i] = v < seen.total ? p : 0xFFFFFFFFu;
      kraw[i] = *reinterpret_cast<const u32x4*>(cache + (size_t)p * s.dp + dc);
      kin[i] = b.kinv[p];
    }
  };
  fetch(rb);
  // this token's norms; its key row where this workgroup has it
  const bool owner = OWN && re == rounds;
  Squares vq, vk;
  squares_fetch(cat + s.off_q, s.heads * s.dim, tid * 4, vq);
  if (owner) squares_fetch(cat + s.off_k, s.kv_heads * s.dim, tid * 4, vk);
  float q[HQ][PER], kn[PER], own[PER], own_inv = 0.0f, slope[HQ];
  const bool vec = (s.dim & 3) == 0;
  auto chunk = [&](const float* p, float* o) { row_chunk<PER>(p, d0, s.dim, vec, o); };   // (values past the head's end: 0)
  chunk(b.kn + g * s.dim, kn);
#pragma unroll
  for (int h = 0; h < HQ; h++) {
    const uint32_t hh = h0 + ((uint32_t)h < hn ? h : 0);
    float w[PER];
    chunk(cat + s.off_q + hh * s.dim, q[h]);
    chunk(b.qn + hh * s.dim, w);
    const float f = s.scale * cap_unit(s.cap) * b.temp[hh];
    slope[h] = tied_slope(hh, s.heads);
#pragma unroll
    for (int e = 0; e < PER; e++) q[h][e] *= w[e] * (kn[e] * f);
  }
  if (owner) {
    chunk(cat + s.off_k + g * s.dim, own);
#pragma unroll
    for (int e = 0; e < PER; e++) own[e] = (float)to_act<T>(own[e]);
  }
  const float sq = squares(cat + s.off_q, s.heads * s.dim, vq), sk = owner ? squares(cat + s.off_k, s.kv_heads * s.dim, vk) : 0.0f;
  const float qinv = 1.0f / __builtin_sqrtf(block_sum(sq, red) / (float)(s.heads * s.dim) + s.eps);
  if (owner) {
    own_inv = 1.0f / __builtin_sqrtf(block_sum(sk, red) / (float)(s.kv_heads * s.dim) + s.eps);
    if (blockIdx.y % chunks == 0 && tid < LPK && d0 < s.dp) {       // the cache row
      T row[PER];
#pragma unroll
      for (int e = 0; e < PER; e++) row[e] = to_act<T>(own[e]);
      __builtin_memcpy(__builtin_assume_aligned(cache + (size_t)pos * s.dp + d0, 16), row, 16);
      if (blockIdx.y == 0 && tid == 0) b.kinv[pos] = own_inv;
    }
  }
#pragma unroll
  for (int h = 0; h < HQ; h++)
#pragma unroll
    for (int e = 0; e < PER; e++) q[h][e] *= qinv;
  const CapF cap(s.cap);
  float m[HQ], l[HQ], o[HQ][PER];
#pragma unroll
  for (int h = 0; h < HQ; h++) {
    m[h] = kTiedNeg; l[h] = 0.0f;
#pragma unroll
    for (int e = 0; e < PER; e++) o[h][e] = 0.0f;
  }
  for (uint32_t r = rb; r < re; r++) {
    u32x4 cur[NB];
    float ci[NB], sc[NB][HQ], bias[NB], top = 0.0f;
    uint32_t cp[NB];
#pragma unroll
    for (int i = 0; i < NB; i++) { cur[i] = kraw[i]; ci[i] = kin[i]; cp[i] = kp[i]; }
    if (r + 1 < re) fetch(r + 1);
    auto row_of = [&](int i, float* kf) {
      unpack_row<T, PER>(cur[i], kf);
      if (OWN && owner && cp[i] == pos) {
#pragma unroll
        for (int e = 0; e < PER; e++) kf[e] = own[e];
      }
    };
#pragma unroll
    for (int i = 0; i < NB; i++) {
      float kf[PER];
      row_of(i, kf);
      const float inv = OWN && owner && cp[i] == pos ? own_inv : ci[i];
      const bool ok = cp[i] != 0xFFFFFFFFu;
      const float dist = (float)(pos - (ok ? cp[i] : pos));
#pragma unroll
      for (int h = 0; h < HQ; h++) {
        float t = 0.0f;
#pragma unroll
        for (int e = 0; e < PER; e++) t = __builtin_fmaf(q[h][e], kf[e], t);
        sc[i][h] = lanes_sum<LPK>(t) * inv;
        top = fmaxf(top, fabsf(sc[i][h]));
      }
      bias[i] = dist;
    }
    if (__any(!(top < cap.lim))) {
      asm volatile("");                        // (kept a branch: scores come near the cap now and then)
#pragma unroll
      for (int i = 0; i < NB; i++)
#pragma unroll
        for (int h = 0; h < HQ; h++) sc[i][h] = cap.any(sc[i][h], -slope[h] * bias[i]);
    } else {
#pragma unroll
      for (int i = 0; i < NB; i++)
#pragma unroll
        for (int h = 0; h < HQ; h++) sc[i][h] = cap.small(sc[i][h], -slope[h] * bias[i]);
    }
#pragma unroll
    for (int i = 0; i < NB; i++)
#pragma unroll
      for (int h = 0; h < HQ; h++) sc[i][h] = cp[i] != 0xFFFFFFFFu ? sc[i][h] : kTiedNeg;
#pragma unroll
    for (int h = 0; h < HQ; h++) {
      float m1 = m[h];
#pragma unroll
      for (int i = 0; i < NB; i++) m1 = fmaxf(m1, sc[i][h]);
      const float a = __builtin_amdgcn_exp2f(m[h] - m1);
      l[h] *= a;
#pragma unroll
      for (int e = 0; e < PER; e++) o[h][e] *= a;
      m[h] = m1;
#pragma unroll
      for (int i = 0; i < NB; i++) {
        const float p = cp[i] != 0xFFFFFFFFu ? __builtin_amdgcn_exp2f(sc[i][h] - m1) : 0.0f;
        sc[i][h] = p;
        l[h] += p;
      }
    }
#pragma unroll
    for (int i = 0; i < NB; i++) {
      float kf[PER];
      row_of(i, kf);
#pragma unroll
      for (int h = 0; h < HQ; h++)
#pragma unroll
        for (int e = 0; e < PER; e++) o[h][e] = __builtin_fmaf(sc[i][h], kf[e], o[h][e]);
    }
  }
  // the key groups' shares: maxima first, then the sums on a common scale
  float mx[HQ];
#pragma unroll
  for (int h = 0; h < HQ; h++) {
    mx[h] = m[h];
#pragma unroll
    for (uint32_t d = LPK; d < 64; d *= 2) mx[h] = fmaxf(mx[h], __shfl_xor(mx[h], d, 64));
    if (lane == 0) ml[0][w][h] = mx[h];
  }
  __syncthreads();
#pragma unroll
  for (int h = 0; h < HQ; h++) {
    mx[h] = fmaxf(fmaxf(ml[0][0][h], ml[0][1][h]), fmaxf(ml[0][2][h], ml[0][3][h]));
    const float a = __builtin_amdgcn_exp2f(m[h] - mx[h]);
    float lw = l[h] * a;
#pragma unroll
    for (uint32_t d = LPK; d < 64; d *= 2) lw += __shfl_xor(lw, d, 64);
    if (lane == 0) ml[1][w][h] = lw;
#pragma unroll
    for (int e = 0; e < PER; e += 4) {
      f32x4 v;
#pragma unroll
      for (int k = 0; k < 4; k++) {
        v[k] = o[h][e + k] * a;
        if constexpr (GPW > 1) v[k] += __shfl_xor(v[k], 32, 64);
      }
      if (lane < HALF) *reinterpret_cast<f32x4*>(accs + ((w * HQ + h) * HALF + lane) * PER + e) = v;
    }
  }
  __syncthreads();
  const size_t rows = (size_t)M * s.heads, r0 = (size_t)sp * rows + (size_t)z * s.heads + h0;
  if (tid < hn) {
    const float lt = (ml[1][0][tid] + ml[1][1][tid]) + (ml[1][2][tid] + ml[1][3][tid]);
    b.part_ml[(r0 + tid) * 2] = mx[0];
    for (uint32_t h = 1; h < (uint32_t)HQ; h++)
      if (tid == h) b.part_ml[(r0 + tid) * 2] = mx[h];
    b.part_ml[(r0 + tid) * 2 + 1] = lt;
  }
  for (uint32_t i = tid; i < hn * s.dim; i += 256) {
    const uint32_t h = i / s.dim, d = i % s.dim, ln = d / PER, e = d % PER;
    float v = 0.0f;
#pragma unroll
    for (uint32_t k = 0; k < 4; k++)
#pragma unroll
      for (uint32_t x = 0; x < HALF; x += LPK) v += accs[((k * HQ + h) * HALF + x + ln) * PER + e];
    b.part_acc[(r0 + h) * s.dim + d] = v;
  }
}

template <class T, uint32_t LPK, int HQ, bool OWN>
static hipError_t tied_attn_go(const TiedShape& s, const TiedBufs& b, const int* pos_ptr, uint32_t pos0, uint32_t M, uint32_t n_splits, hipStream_t st) {
  const uint32_t gq = s.heads / s.kv_heads, chunks = (gq + HQ - 1) / HQ;
  const size_t lds = (size_t)4 * HQ * (64 / LPK > 1 ? 32 : 64) * (16 / sizeof(T)) * 4;
  hipLaunchKernelGGL((tied_attn_kernel<T, LPK, HQ, OWN>), dim3(n_splits, s.kv_heads * chunks, M), dim3(256), lds, st, s, b, pos_ptr, pos0, M, n_splits);
  return hipGetLastError();
}
template <class T, uint32_t LPK>
static hipError_t tied_attn_pick(const TiedShape& s, const TiedBufs& b, const int* pos_ptr, uint32_t pos0, uint32_t M, bool own, uint32_t n_splits, hipStream_t st) {
  const uint32_t gq = s.heads / s.kv_heads;
#define LGH_TIED_CASE(N) return own ? tied_attn_go<T, LPK, N, true>(s, b, pos_ptr, pos0, M, n_splits, st) : tied_attn_go<T, LPK, N, false>(s, b, pos_ptr, pos0, M, n_splits, st)
  if (gq == 1) LGH_TIED_CASE(1);
  if (gq == 2) LGH_TIED_CASE(2);
  LGH_TIED_CASE(4);
#undef LGH_TIED_CASE
}
static bool tied_ok(const TiedShape& s) {
  return s.heads && s.kv_heads && s.heads % s.kv_heads == 0 && s.dim && s.dim <= s.dp && s.dp % 64 == 0 && s.dp <= kTiedMaxDim && s.window && s.rows % 64 == 0;
}

hipError_t tied_attn_launch(const TiedShape& s, const TiedBufs& b, const int* pos_ptr, uint32_t pos0, uint32_t M, bool own, uint32_t n_splits, bool f32, hipStream_t st) {
  if (!tied_ok(s) || M == 0 || M > kTiedShort || (own && M != 1) || n_splits == 0 || n_splits > kTiedMaxSplits || (!pos_ptr && pos0 + M > s.rows)) return hipErrorInvalidValue;
  switch (tied_lanes(s.dp, f32 ? 4 : 2)) {
    case 8: return f32 ? hipErrorInvalidValue : tied_attn_pick<__bf16, 8>(s, b, pos_ptr, pos0, M, own, n_splits, st);
    case 16: return f32 ? tied_attn_pick<float, 16>(s, b, pos_ptr, pos0, M, own, n_splits, st) : tied_attn_pick<__bf16, 16>(s, b, pos_ptr, pos0, M, own, n_splits, st);
    case 32: return f32 ? tied_attn_pick<float, 32>(s, b, pos_ptr, pos0, M, own, n_splits, st) : tied_attn_pick<__bf16, 32>(s, b, pos_ptr, pos0, M, own, n_splits, st);
    case 64: return f32 ? tied_attn_pick<float, 64>(s, b, pos_ptr, pos0, M, own, n_splits, st) : hipErrorInvalidValue;
  }
  return hipErrorInvalidValue;
}

uint32_t tied_keys_per_round(const TiedShape& s, bool f32) { return tied_round(tied_lanes(s.dp, f32 ? 4 : 2)); }

// shares of the keys that fill the chip; not more than there are rounds of keys
uint32_t tied_splits(const TiedShape& s, uint32_t max_seq, uint32_t M, bool f32, uint32_t forced) {
  const uint32_t gq = s.heads / s.kv_heads, hq = gq <= 2 ? gq : 4, wgs = s.kv_heads * ((gq + hq - 1) / hq) * M;
  const uint32_t kr = tied_keys_per_round(s, f32), rounds = (tied_seen(s, max_seq - 1).total + kr - 1) / kr;
  const uint32_t want = forced ? forced : std::max(1u, 512 / wgs);
  return std::min(std::min(want, kTiedMaxSplits), std::max(rounds, 1u));
}

// the shares of the keys put together, the sink's term; grid (heads, tokens).  V: 4 where heads have a multiple of 4 values
template <class O, int V>
__global__ void __launch_bounds__(256) tied_merge_kernel(const TiedShape s, const TiedBufs b, const int* __restrict__ pos_ptr, uint32_t pos0, uint32_t M, uint32_t n_splits,
                                                         uint32_t kr, O* __restrict__ out, uint32_t ldo) {
  struct Val { float v[V]; };
  __shared__ Val part[256];
  __shared__ float wgt[kTiedMaxSplits];
  static_assert(kTiedMaxSplits == 128, "two splits per lane");
  const uint32_t tid = threadIdx.x, lane = tid & 63, h = blockIdx.x, t = blockIdx.y;
  const uint32_t pos = (pos_ptr ? (uint32_t)*pos_ptr : pos0) + t;
  const uint32_t rounds = (tied_seen(s, pos).total + kr - 1) / kr, per = (rounds + n_splits - 1) / n_splits, act = (rounds + per - 1) / per;
  const size_t rows = (size_t)M * s.heads, r = (size_t)t * s.heads + h;
  // (what the inactive shares hold is not used: the loads need no position)
  f32x2 ml[2];
#pragma unroll
  for (uint32_t k = 0; k < 2; k++) {
    const uint32_t i = lane + k * 64;
    ml[k] = *reinterpret_cast<const f32x2*>(b.part_ml + ((i < n_splits ? i : n_splits - 1) * rows + r) * 2);
  }
  const float sink = b.sink[h] * kTiedLog2e;
  // columns x groups of splits; the first partial sums are requested before the weights are known
  const uint32_t cols = (s.dim + V - 1) / V, groups = 256 / cols, grp = tid / cols, c0 = tid % cols * V;
  auto load = [&](uint32_t k) {
    Val x;
    const float* p = b.part_acc + (k * rows + r) * s.dim + c0;
    if constexpr (V == 4) { const f32x4 q = *reinterpret_cast<const f32x4*>(p); x.v[0] = q.x; x.v[1] = q.y; x.v[2] = q.z; x.v[3] = q.w; }
    else x.v[0] = p[0];
    return x;
  };
  constexpr int F = 8;
  Val first[F], v;
#pragma unroll
  for (int i = 0; i < F; i++) first[i] = load(grp + i * groups < n_splits ? grp + i * groups : n_splits - 1);
  if (tid < 64) {
    const float m0 = lane < act ? ml[0].x : kTiedNeg, m1 = lane + 64 < act ? ml[1].x : kTiedNeg;
    const float mm = fmaxf(wave_max(fmaxf(m0, m1)), sink);
    const float f0 = __builtin_amdgcn_exp2f(m0 - mm), f1 = __builtin_amdgcn_exp2f(m1 - mm);
    const float l0 = lane < act ? f0 * ml[0].y : 0.0f, l1 = lane + 64 < act ? f1 * ml[1].y : 0.0f;
    const float tot = wave_sum(l0 + l1) + __builtin_amdgcn_exp2f(sink - mm);
    wgt[lane] = f0 / tot; wgt[lane + 64] = f1 / tot;
  }
  __syncthreads();
#pragma unroll
  for (int j = 0; j < V; j++) v.v[j] = 0.0f;
  if (grp < groups) {
#pragma unroll
    for (int i = 0; i < F; i++) {
      const uint32_t k = grp + i * groups;
      if (k < act)
#pragma unroll
        for (int j = 0; j < V; j++) v.v[j] = __builtin_fmaf(wgt[k], first[i].v[j], v.v[j]);
    }
    for (uint32_t k = grp + F * groups; k < act; k += groups) {
      const Val x = load(k);
#pragma unroll
      for (int j = 0; j < V; j++) v.v[j] = __builtin_fmaf(wgt[k], x.v[j], v.v[j]);
    }
  }
  part[tid] = v;
  __syncthreads();
  if (tid < cols) {
    for (uint32_t k = 1; k < groups; k++)
#pragma unroll
      for (int j = 0; j < V; j++) v.v[j] += part[tid + k * cols].v[j];
#pragma unroll
    for (int j = 0; j < V; j++) out[(size_t)t * ldo + h * s.dim + c0 + j] = to_act<O>(v.v[j]);
  }
}

hipError_t tied_merge_launch(const TiedShape& s, const TiedBufs& b, const int* pos_ptr, uint32_t pos0, uint32_t M, uint32_t n_splits, bool f32, void* out, uint32_t ldo,
                             bool out_f32, hipStream_t st) {
  if (!tied_ok(s) || n_splits == 0 || n_splits > kTiedMaxSplits || M == 0) return hipErrorInvalidValue;
  const uint32_t kr = tied_keys_per_round(s, f32);
  const dim3 grid(s.heads, M);
  const bool v4 = s.dim % 4 == 0;
  if (out_f32 && v4) hipLaunchKernelGGL((tied_merge_kernel<float, 4>), grid, dim3(256), 0, st, s, b, pos_ptr, pos0, M, n_splits, kr, (float*)out, ldo);
  else if (out_f32) hipLaunchKernelGGL((tied_merge_kernel<float, 1>), grid, dim3(256), 0, st, s, b, pos_ptr, pos0, M, n_splits, kr, (float*)out, ldo);
  else if (v4) hipLaunchKernelGGL((tied_merge_kernel<__bf16, 4>), grid, dim3(256), 0, st, s, b, pos_ptr, pos0, M, n_splits, kr, (__bf16*)out, ldo);
  else hipLaunchKernelGGL((tied_merge_kernel<__bf16, 1>), grid, dim3(256), 0, st, s, b, pos_ptr, pos0, M, n_splits, kr, (__bf16*)out, ldo);
  return hipGetLastError();
}

// a block's cache rows, key factors and queries; grid (tokens).  V: 4 where heads have a multiple of 4 values
template <class T, int V>
__global__ void __launch_bounds__(256) tied_prep_kernel(const TiedShape s, const TiedBufs b, uint32_t pos0) {
  __shared__ float red[16];
  const uint32_t t = blockIdx.x, pos = pos0 + t, tid = threadIdx.x, nq = s.heads * s.dim, nk = s.kv_heads * s.dim, gq = s.heads / s.kv_heads;
  const float* cat = b.cat + (size_t)t * s.ldcat;
  struct Val { float v[V]; };
  auto load = [](const float* p) {
    Val r;
    if constexpr (V == 4) { const f32x4 q = *reinterpret_cast<const f32x4*>(p); r.v[0] = q.x; r.v[1] = q.y; r.v[2] = q.z; r.v[3] = q.w; }
    else r.v[0] = p[0];
    return r;
  };
  auto store = [](T* p, const Val& a) {
    T o[V];
#pragma unroll
    for (int i = 0; i < V; i++) o[i] = to_act<T>(a.v[i]);
    __builtin_memcpy(__builtin_assume_aligned(p, sizeof(o)), o, sizeof(o));
  };
  Squares vq, vk;
  squares_fetch(cat + s.off_q, nq, tid * 4, vq);
  squares_fetch(cat + s.off_k, nk, tid * 4, vk);
  for (uint32_t i = tid * V; i < nk; i += 256 * V)
    store(reinterpret_cast<T*>(b.cache) + ((size_t)(i / s.dim) * s.rows + pos) * s.dp + i % s.dim, load(cat + s.off_k + i));
  const float sk = squares(cat + s.off_k, nk, vk), sq = squares(cat + s.off_q, nq, vq);
  const float kinv = 1.0f / __builtin_sqrtf(block_sum(sk, red) / (float)nk + s.eps);
  if (tid == 0) b.kinv[pos] = kinv;
  if (!b.q) return;
  const float qinv = 1.0f / __builtin_sqrtf(block_sum(sq, red) / (float)nq + s.eps) * s.scale * cap_unit(s.cap);
  for (uint32_t i = tid * V; i < s.heads * s.dp; i += 256 * V) {
    const uint32_t h = i / s.dp, d = i % s.dp, dd = d < s.dim ? d : 0;
    const Val q = load(cat + s.off_q + h * s.dim + dd), qn = load(b.qn + h * s.dim + dd), kn = load(b.kn + h / gq * s.dim + dd);
    const float f = d < s.dim ? qinv * b.temp[h] : 0.0f;
    Val o;
#pragma unroll
    for (int e = 0; e < V; e++) o.v[e] = q.v[e] * qn.v[e] * (kn.v[e] * f);
    store(reinterpret_cast<T*>(b.q) + ((size_t)h * b.Mcap + t) * s.dp + d, o);
  }
}

hipError_t tied_prep_launch(const TiedShape& s, const TiedBufs& b, uint32_t pos0, uint32_t M, bool f32, hipStream_t st) {
  if (!tied_ok(s) || M == 0 || (b.q && M > b.Mcap) || pos0 + M > s.rows) return hipErrorInvalidValue;
  const bool v4 = s.dim % 4 == 0;
  if (f32 && v4) hipLaunchKernelGGL((tied_prep_kernel<float, 4>), dim3(M), dim3(256), 0, st, s, b, pos0);
  else if (f32) hipLaunchKernelGGL((tied_prep_kernel<float, 1>), dim3(M), dim3(256), 0, st, s, b, pos0);
  else if (v4) hipLaunchKernelGGL((tied_prep_kernel<__bf16, 4>), dim3(M), dim3(256), 0, st, s, b, pos0);
  else hipLaunchKernelGGL((tied_prep_kernel<__bf16, 1>), dim3(M), dim3(256), 0, st, s, b, pos0);
  return hipGetLastError();
}

// ------------------------------------------------------------------------------------------------
// prompt portions.  A workgroup = 4 waves = 64 * QT queries of one head; S^T = K Q^T leaves a lane with one query's scores of keys
// 4g .. 4g + 3, which is the operand of O^T = K^T P^T, whose key fragments come out of the same LDS tile by transposed reads.  Tiles of KT
// keys go to LDS by DMA, two buffers: first the kept tiles in front of the window, then the tiles from the first query's window on.
// ------------------------------------------------------------------------------------------------
template <class T> constexpr int tied_kt() { return sizeof(T) == 2 ? 64 : 32; }
template <class T, int DQ> constexpr size_t tied_lds() { return 2 * (size_t)tied_kt<T>() * DQ * sizeof(T); }
template <class T, int DQ> constexpr int tied_qt() { return sizeof(T) == 2 && DQ <= 192 ? 2 : 1; }   // 16-query tiles per wave
template <class T, int DQ> constexpr int tied_wgs() { return DQ <= 128 ? 2 : 1; }

template <class T, int DQ>
__global__ void __launch_bounds__(256, (tied_wgs<T, DQ>())) tied_flash_kernel(const TiedShape s, const TiedBufs b, uint32_t pos0, uint32_t M, uint32_t nqb, T* __restrict__ out,
                                                                              uint32_t ldo) {
  constexpr bool BF = sizeof(T) == 2;
  constexpr int KT = tied_kt<T>(), QT = tied_qt<T, DQ>(), NK = KT / 16, NU = DQ / Frag<T>::KU, ND = DQ / 16;
  constexpr uint32_t XC = DQ * sizeof(T) / 16, kBuf = KT * XC * 16;
  extern __shared__ __attribute__((aligned(16))) uint8_t smem[];
  const uint32_t lane = threadIdx.x & 63, w = (uint32_t)__builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6)), r16 = lane & 15, g = lane >> 4;
  // the longest rows first, and of the second half of the grid the shortest first (workgroups i and i + half share a CU when all are resident)
  const uint32_t h = blockIdx.x % s.heads, qi = blockIdx.x / s.heads, hi = (nqb + 1) / 2, qb = qi < hi ? nqb - 1 - qi : qi - hi;
  const uint32_t q0 = qb * 64 * QT, qw = q0 + w * 16 * QT, qlast = q0 + 64 * QT - 1 < M - 1 ? q0 + 64 * QT - 1 : M - 1;
  const uint32_t ifirst = pos0 + q0, lo = ifirst + 1 > s.window ? ifirst + 1 - s.window : 0, tw = lo / KT;
  const uint32_t kt = (s.keep + KT - 1) / KT, nkt = kt < tw ? kt : tw;                // kept tiles in front of the window's first one
  const uint32_t tiles = nkt + (pos0 + qlast) / KT + 1 - tw;
  const T* K = reinterpret_cast<const T*>(b.cache) + (size_t)(h / (s.heads / s.kv_heads)) * s.rows * DQ;
  const uint32_t lds0 = (uint32_t)__builtin_amdgcn_readfirstlane((int)lds_addr_of(smem));
  auto tile_at = [&](uint32_t i) { return i < nkt ? i : tw + i - nkt; };
  auto stage = [&](uint32_t tl, uint32_t buf) {
#pragma unroll
    for (int i = 0; i < (int)(kBuf / 4096); i++) {
      const uint32_t c = (i * 4 + w) * 64 + lane, row = c / XC, ch = (c % XC) ^ (row & 7);
      lds_dma16_untracked(K + ((size_t)tl * KT + row) * DQ + ch * (16 / sizeof(T)), lds0 + buf * kBuf + (i * 4 + w) * 1024);
    }
  };
  f32x4 kin[NK];
  auto factors = [&](uint32_t tl) {
#pragma unroll
    for (int n = 0; n < NK; n++) kin[n] = *reinterpret_cast<const f32x4*>(b.kinv + (size_t)tl * KT + n * 16 + g * 4);
  };
  factors(tile_at(0));
  stage(tile_at(0), 0);
  typename Frag<T>::V qf[QT][NU];
#pragma unroll
  for (int t = 0; t < QT; t++) {
    const uint32_t m = qw + t * 16 + r16;
    const T* qr = reinterpret_cast<const T*>(b.q) + ((size_t)h * b.Mcap + (m < M ? m : M - 1)) * DQ + g * Frag<T>::PER;
#pragma unroll
    for (int u = 0; u < NU; u++) qf[t][u] = Frag<T>::load(qr + u * Frag<T>::KU);
  }
  f32x4 o[ND][QT];
  float mx[QT], l[QT];
#pragma unroll
  for (int t = 0; t < QT; t++) {
    mx[t] = kTiedNeg; l[t] = 0.0f;
#pragma unroll
    for (int i = 0; i < ND; i++) o[i][t] = (f32x4)(0.0f);
  }
  const CapF cap(s.cap);
  const float slope = tied_slope(h, s.heads);
  f32x4 bias[NK];                                               // slope * (place in the tile) of this lane's keys
#pragma unroll
  for (int n = 0; n < NK; n++)
#pragma unroll
    for (int e = 0; e < 4; e++) bias[n][e] = slope * (float)(n * 16 + g * 4 + e);
  const uint32_t iw0 = pos0 + qw, iw1 = iw0 + 16 * QT - 1;      // this wave's queries
  wait_vm(0);
  __syncthreads();
  for (uint32_t it = 0; it < tiles; it++) {
    const uint32_t cur = it & 1, k0 = tile_at(it) * KT, k1 = k0 + KT - 1;
    f32x4 kc[NK];
#pragma unroll
    for (int n = 0; n < NK; n++) kc[n] = kin[n];
    if (it + 1 < tiles) {
      factors(tile_at(it + 1));
      stage(tile_at(it + 1), cur ^ 1);
    }
    // (wave-uniform) no query of this wave sees the tile / every one sees all of it
    const bool none = k0 > iw1 || (iw0 > k1 && iw0 - k1 >= s.window && k0 >= s.keep);
    const bool full = k1 <= iw0 && (iw1 - k0 < s.window || k1 < s.keep);
    if (!none) {
      const T* tile = reinterpret_cast<const T*>(smem + cur * kBuf);
      f32x4 sa[NK][QT];
#pragma unroll
      for (int n = 0; n < NK; n++)
#pragma unroll
        for (int t = 0; t < QT; t++) sa[n][t] = (f32x4)(0.0f);
      __builtin_amdgcn_s_setprio(1);   // products ahead of the other waves' softmax
#pragma unroll
      for (int u = 0; u < NU; u++)
#pragma unroll
        for (int n = 0; n < NK; n++) {
          const uint32_t row = n * 16 + r16;
          const typename Frag<T>::V kf = Frag<T>::load(tile + row * DQ + (((uint32_t)(u * 4) + g) ^ (row & 7)) * Frag<T>::PER);
#pragma unroll
          for (int t = 0; t < QT; t++) sa[n][t] = Frag<T>::mma(kf, qf[t][u], sa[n][t]);
        }
      __builtin_amdgcn_s_setprio(0);
      float top = 0.0f;
#pragma unroll
      for (int t = 0; t < QT; t++)
#pragma unroll
        for (int n = 0; n < NK; n++)
#pragma unroll
          for (int e = 0; e < 4; e++) {
            sa[n][t][e] *= kc[n][e];
            top = fmaxf(top, fabsf(sa[n][t][e]));
          }
      if (__any(!(top < cap.lim))) {
        asm volatile("");              // (kept a branch: scores come near the cap now and then)
#pragma unroll
        for (int t = 0; t < QT; t++)
#pragma unroll
          for (int n = 0; n < NK; n++)
#pragma unroll
            for (int e = 0; e < 4; e++) sa[n][t][e] = cap.any(sa[n][t][e], bias[n][e]);
      } else {
#pragma unroll
        for (int t = 0; t < QT; t++)
#pragma unroll
          for (int n = 0; n < NK; n++)
#pragma unroll
            for (int e = 0; e < 4; e++) sa[n][t][e] = BF ? cap.small_bf(sa[n][t][e], bias[n][e]) : cap.small(sa[n][t][e], bias[n][e]);
      }
#pragma unroll
      for (int t = 0; t < QT; t++) {
        const uint32_t i = iw0 + t * 16 + r16;
        const float off = slope * (float)(int)(k0 - i);      // what the tile's place adds to every score of this lane's query
        if (!full) {
          asm volatile("");              // (kept a branch: most tiles have no masks to apply)
#pragma unroll
          for (int n = 0; n < NK; n++)
#pragma unroll
            for (int e = 0; e < 4; e++) {
              const uint32_t j = k0 + n * 16 + g * 4 + e;
              sa[n][t][e] = j <= i && (i - j < s.window || j < s.keep) ? sa[n][t][e] : kTiedNeg;
            }
        }
        float m1 = kTiedNeg;
#pragma unroll
        for (int n = 0; n < NK; n++)
#pragma unroll
          for (int e = 0; e < 4; e++) m1 = fmaxf(m1, sa[n][t][e]);
        m1 = fmaxf(m1, __shfl_xor(m1, 16, 64));
        m1 = fmaxf(m1, __shfl_xor(m1, 32, 64)) + off;
        // the reference follows the maximum once it has risen by more than 2^8: weights stay far from overflow, most tiles rescale nothing; each
        // query by itself, so that its rounding does not depend on its neighbours
        // (a query that has seen nothing yet weighs masked keys; the factor of its first visible tile takes that to 0)
        if (__any(m1 > mx[t] + 8.0f)) {
          asm volatile("");
          const float m2 = m1 > mx[t] + 8.0f ? m1 : mx[t], a = __builtin_amdgcn_exp2f(mx[t] - m2);
          mx[t] = m2;
          l[t] *= a;
#pragma unroll
          for (int d = 0; d < ND; d++) o[d][t] *= a;
        }
        const float rel = mx[t] - off;
        float sum = 0.0f;
#pragma unroll
        for (int n = 0; n < NK; n++)
#pragma unroll
          for (int e = 0; e < 4; e++) {
            const float p = __builtin_amdgcn_exp2f(sa[n][t][e] - rel);
            sa[n][t][e] = p;
            sum += p;
          }
        l[t] += sum;
      }
      __builtin_amdgcn_s_setprio(1);
      if constexpr (BF) {
#pragma unroll
        for (int u = 0; u < KT / 32; u++) {
          bf16x8 pf[QT];
#pragma unroll
          for (int t = 0; t < QT; t++)
#pragma unroll
            for (int e = 0; e < 4; e++) { pf[t][e] = (__bf16)sa[2 * u][t][e]; pf[t][4 + e] = (__bf16)sa[2 * u + 1][t][e]; }
#pragma unroll
          for (int d = 0; d < ND; d++) {
            const bf16x8 vf = tile_value_frag<T>(tile + u * 32 * DQ, DQ, 0, d * 16, r16, g);
#pragma unroll
            for (int t = 0; t < QT; t++) o[d][t] = Frag<T>::mma(vf, pf[t], o[d][t]);
          }
        }
      } else {
#pragma unroll
        for (int n = 0; n < NK; n++)
#pragma unroll
          for (int d = 0; d < ND; d++) {
            const f32x4 vf = tile_value_frag<T>(tile, DQ, n, d * 16, r16, g);
#pragma unroll
            for (int t = 0; t < QT; t++) o[d][t] = Frag<T>::mma(vf, sa[n][t], o[d][t]);
          }
      }
      __builtin_amdgcn_s_setprio(0);
    }
    wait_vm(0);
    __syncthreads();
  }
  const float sink = b.sink[h] * kTiedLog2e;
#pragma unroll
  for (int t = 0; t < QT; t++) {
    float lt = l[t];
    lt += __shfl_xor(lt, 16, 64);
    lt += __shfl_xor(lt, 32, 64);
    const uint32_t m = qw + t * 16 + r16;
    if (m >= M) continue;
    const float mm = fmaxf(mx[t], sink), a = __builtin_amdgcn_exp2f(mx[t] - mm), fac = a / (lt * a + __builtin_amdgcn_exp2f(sink - mm));
    T* dst = out + (size_t)m * ldo + h * s.dim;
#pragma unroll
    for (int d = 0; d < ND; d++)
#pragma unroll
      for (int e = 0; e < 4; e++) {
        const uint32_t v = d * 16 + g * 4 + e;
        if (v < s.dim) dst[v] = to_act<T>(o[d][t][e] * fac);
      }
  }
}

template <class T, int DQ>
static hipError_t tied_flash_go(const TiedShape& s, const TiedBufs& b, uint32_t pos0, uint32_t M, void* out, uint32_t ldo, hipStream_t st) {
  static bool opted[64] = {};
  constexpr size_t lds = tied_lds<T, DQ>();
  static_assert(lds <= 160 * 1024, "two tiles fit LDS");
  if (hipError_t e = lds_opt_in(reinterpret_cast<const void*>(&tied_flash_kernel<T, DQ>), (int)lds, opted); e != hipSuccess) return e;
  const uint32_t QB = 64 * tied_qt<T, DQ>(), nqb = (M + QB - 1) / QB;
  hipLaunchKernelGGL((tied_flash_kernel<T, DQ>), dim3(nqb * s.heads), dim3(256), lds, st, s, b, pos0, M, nqb, (T*)out, ldo);
  return hipGetLastError();
}

hipError_t tied_flash_launch(const TiedShape& s, const TiedBufs& b, uint32_t pos0, uint32_t M, bool f32, void* out, uint32_t ldo, hipStream_t st) {
  if (!tied_ok(s) || !b.q || M == 0 || M > b.Mcap || (uint64_t)(pos0 + M + 63) / 64 * 64 > s.rows) return hipErrorInvalidValue;   // whole key tiles are read
#define LGH_FLASH_CASE(Q) if (s.dp == Q) return f32 ? tied_flash_go<float, Q>(s, b, pos0, M, out, ldo, st) : tied_flash_go<__bf16, Q>(s, b, pos0, M, out, ldo, st);
  LGH_FLASH_CASE(64) LGH_FLASH_CASE(128) LGH_FLASH_CASE(192) LGH_FLASH_CASE(256)
#undef LGH_FLASH_CASE
  return hipErrorInvalidValue;
}

}  // namespace lgh
