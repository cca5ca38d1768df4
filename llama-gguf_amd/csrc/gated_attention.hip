// gated_attention.hip — grouped softmax attention of layered.h with values of their own size: queries and keys are (RMS-normed per head and) rotated
// (neighbouring pairs) before they are used or cached, position i sees the keys of its own chunk (counted from the sequence's start) and of its window
// up to itself, the softmax may have a sink (one more term exp(0), which has no value), and the heads' outputs may be gated value by value.  Scores,
// softmax and sums are in 32-bit, in units of log2.
//
//   decode and short portions: a workgroup = one key head (up to 4 of its query heads) x one share of the visible keys; a lane holds 16-byte
//     pieces of a few keys' and values' rows, for the score and for the weighted sum.  In decode the same launch steps the gated linear attention
//     that reads the same input (further workgroups), and the merge of the shares reads it out.
//   prompt portions: causal flash attention in transposed form (S^T = K Q^T, O^T = V^T P^T), key and value tiles through LDS; only the tiles
//     from the first query's first visible key on.
// A layer may read another layer's caches: it has queries only, and its launches come after the ones that fill them.
#include <algorithm>

#include "gla_device.h"

namespace lgh {

constexpr float kGattnNeg = -1e30f, kGattnLog2e = 1.4426950408889634f;
constexpr uint32_t kGattnMaxSplits = 128, kGattnBatch = 4;

// the first key that position i sees; never falls with i
__host__ __device__ __forceinline__ uint32_t key_start(const GattnShape& s, uint32_t i) {
  const uint32_t c = i / s.chunk * s.chunk, w = i >= s.window ? i - s.window + 1 : 0;
  return c > w ? c : w;
}

// lanes that share a row: 16 bytes each, of the wider of key and value
__host__ __device__ constexpr uint32_t gattn_lanes(uint32_t bytes) { return bytes <= 128 ? 8 : bytes <= 256 ? 16 : bytes <= 512 ? 32 : 64; }
__host__ __device__ constexpr uint32_t gattn_round(uint32_t lanes) { return 4 * kGattnBatch * (64 / lanes); }   // keys of a workgroup per round
static uint32_t gattn_row_bytes(const GattnShape& s, bool f32) { return std::max(s.dp, s.vp) * (f32 ? 4 : 2); }

// factor of a pair's rotation
__device__ __forceinline__ f32x2 rotate2(float u, float v, f32x2 cs) {
  f32x2 r;
  r.x = u * cs.x - v * cs.y;
  r.y = v * cs.x + u * cs.y;
  return r;
}

// ------------------------------------------------------------------------------------------------
// decode and short portions; grid: x = (split, key head x chunk of HQ query heads), then the linear attention's workgroups; y = token.
// C: 16-byte pieces per lane and row (2 where 64 lanes do not cover a row)
// ------------------------------------------------------------------------------------------------
template <class T, uint32_t LPK, int HQ, int C, bool OWN>
__device__ __forceinline__ void gattn_split(const GattnShape& s, const GattnBufs& b, uint32_t pos, uint32_t z, uint32_t M, uint32_t sp, uint32_t hy, uint32_t n_splits, float* accs) {
  constexpr int PER = 16 / sizeof(T), NB = kGattnBatch;
  constexpr uint32_t GPW = 64 / LPK, HALF = GPW > 1 ? 32 : 64;      // key groups of a wave; lanes left after folding its halves
  __shared__ float ml[2][4][HQ];
  const uint32_t tid = threadIdx.x, lane = tid & 63, w = tid >> 6, grp = lane / LPK, sub = lane % LPK;
  const uint32_t gq = s.heads / s.kv_heads, chunks = (gq + HQ - 1) / HQ, g = hy / chunks, h0 = g * gq + (hy % chunks) * HQ;
  const uint32_t hn = (g + 1) * gq - h0 < (uint32_t)HQ ? (g + 1) * gq - h0 : (uint32_t)HQ;
  const uint32_t lo = key_start(s, pos), total = pos + 1 - lo;
  constexpr uint32_t KR = gattn_round(LPK);
  const uint32_t rounds = (total + KR - 1) / KR, per = (rounds + n_splits - 1) / n_splits;
  const uint32_t rb = sp * per, re = rb + per < rounds ? rb + per : rounds;
  if (rb >= re) return;                                             // (the merge skips the same splits)
  const float* cat = b.cat + (size_t)z * s.ldcat;
  T* kc = reinterpret_cast<T*>(b.kc) + (size_t)g * s.rows * s.dp;
  T* vc = reinterpret_cast<T*>(b.vc) + (size_t)g * s.rows * s.vp;
  uint32_t d0[C], dk[C], dv[C];
#pragma unroll
  for (int c = 0; c < C; c++) {
    d0[c] = (c * LPK + sub) * PER;
    dk[c] = d0[c] < s.dp ? d0[c] : 0;
    dv[c] = d0[c] < s.vp ? d0[c] : 0;
  }
  u32x4 kraw[NB][C], vraw[NB][C];
  uint32_t kp[NB];
  auto fetch = [&](uint32_t r) {
#pragma unroll
    for (int i = 0; i < NB; i++) {
      const uint32_t v = (r * 4 + w) * (NB * GPW) + i * GPW + grp, p = lo + (v < total ? v : total - 1);
      kp[i] = v < total ? p : 0xFFFFFFFFu;
#pragma unroll
      for (int c = 0; c < C; c++) {
        kraw[i][c] = *reinterpret_cast<const u32x4*>(kc + (size_t)p * s.dp + dk[c]);
        vraw[i][c] = *reinterpret_cast<const u32x4*>(vc + (size_t)p * s.vp + dv[c]);
      }
    }
  };
  fetch(rb);
  // a head's row of this token: normed, rotated.  Everything the rows need is requested before the first of them is used.
  const bool owner = OWN && re == rounds, kvec = (s.dim & 3) == 0, vvec = (s.vdim & 3) == 0, normed = b.qn != nullptr;
  float q[HQ][C][PER], ok[C][PER], ov[C][PER], nq[C][PER], nk[C][PER];
  f32x2 cs[C][PER / 2];
#pragma unroll
  for (int c = 0; c < C; c++) {
    if (normed) row_chunk<PER>(b.qn, d0[c], s.dim, kvec, nq[c]);
#pragma unroll
    for (int h = 0; h < HQ; h++) row_chunk<PER>(cat + s.off_q + (size_t)(h0 + ((uint32_t)h < hn ? h : 0)) * s.dim, d0[c], s.dim, kvec, q[h][c]);
#pragma unroll
    for (int e = 0; e < PER / 2; e++) {
      const uint32_t d = d0[c] + 2 * e;
      cs[c][e].x = 1.0f; cs[c][e].y = 0.0f;
      if (d < s.rot_n) cs[c][e] = reinterpret_cast<const f32x2*>(b.cs)[(size_t)pos * (s.rot_n / 2) + d / 2];
    }
    if (owner) {
      if (normed) row_chunk<PER>(b.kn, d0[c], s.dim, kvec, nk[c]);
      row_chunk<PER>(cat + s.off_k + (size_t)g * s.dim, d0[c], s.dim, kvec, ok[c]);
      row_chunk<PER>(cat + s.off_v + (size_t)g * s.vdim, d0[c], s.vdim, vvec, ov[c]);
    }
  }
  auto head_row = [&](float (*o)[PER], const float (*nf)[PER], float f) {
    if (normed) {
      float ss = 0.0f;
#pragma unroll
      for (int c = 0; c < C; c++)
#pragma unroll
        for (int e = 0; e < PER; e++) ss = __builtin_fmaf(o[c][e], o[c][e], ss);
      const float inv = 1.0f / __builtin_sqrtf(lanes_sum<LPK>(ss) / (float)s.dim + s.eps);
#pragma unroll
      for (int c = 0; c < C; c++)
#pragma unroll
        for (int e = 0; e < PER; e++) o[c][e] *= inv * nf[c][e];
    }
#pragma unroll
    for (int c = 0; c < C; c++)
#pragma unroll
      for (int e = 0; e < PER; e += 2) {
        const f32x2 r = rotate2(o[c][e] * f, o[c][e + 1] * f, cs[c][e / 2]);
        o[c][e] = r.x; o[c][e + 1] = r.y;
      }
  };
#pragma unroll
  for (int h = 0; h < HQ; h++) head_row(q[h], nq, s.scale * kGattnLog2e);
  if (owner) {
    head_row(ok, nk, 1.0f);
#pragma unroll
    for (int c = 0; c < C; c++) {
      T rk[PER], rv[PER];
#pragma unroll
      for (int e = 0; e < PER; e++) {
        rk[e] = to_act<T>(ok[c][e]);
        rv[e] = to_act<T>(ov[c][e]);
        ok[c][e] = (float)rk[e];
        ov[c][e] = (float)rv[e];
      }
      if (hy % chunks == 0 && tid < LPK) {                          // the cache rows
        if (d0[c] < s.dp) __builtin_memcpy(__builtin_assume_aligned(kc + (size_t)pos * s.dp + d0[c], 16), rk, 16);
        if (d0[c] < s.vp) __builtin_memcpy(__builtin_assume_aligned(vc + (size_t)pos * s.vp + d0[c], 16), rv, 16);
      }
    }
  }
  float m[HQ], l[HQ], o[HQ][C][PER];
#pragma unroll
  for (int h = 0; h < HQ; h++) {
    m[h] = kGattnNeg; l[h] = 0.0f;
#pragma unroll
    for (int c = 0; c < C; c++)
#pragma unroll
      for (int e = 0; e < PER; e++) o[h][c][e] = 0.0f;
  }
  for (uint32_t r = rb; r < re; r++) {
    u32x4 ck[NB][C], cv[NB][C];
    float sc[NB][HQ];
    uint32_t cp[NB];
#pragma unroll
    for (int i = 0; i < NB; i++) {
      cp[i] = kp[i];
#pragma unroll
      for (int c = 0; c < C; c++) { ck[i][c] = kraw[i][c]; cv[i][c] = vraw[i][c]; }
    }
    if (r + 1 < re) fetch(r + 1);
#pragma unroll
    for (int i = 0; i < NB; i++) {
      const bool own = OWN && owner && cp[i] == pos;
      float t[HQ];
#pragma unroll
      for (int h = 0; h < HQ; h++) t[h] = 0.0f;
#pragma unroll
      for (int c = 0; c < C; c++) {
        float kf[PER];
        unpack_row<T, PER>(ck[i][c], kf);
#pragma unroll
        for (int e = 0; e < PER; e++) kf[e] = own ? ok[c][e] : kf[e];
#pragma unroll
        for (int h = 0; h < HQ; h++)
#pragma unroll
          for (int e = 0; e < PER; e++) t[h] = __builtin_fmaf(q[h][c][e], kf[e], t[h]);
      }
#pragma unroll
      for (int h = 0; h < HQ; h++) {
        const float v = lanes_sum<LPK>(t[h]);
        sc[i][h] = cp[i] != 0xFFFFFFFFu ? v : kGattnNeg;
      }
    }
#pragma unroll
    for (int h = 0; h < HQ; h++) {
      float m1 = m[h];
#pragma unroll
      for (int i = 0; i < NB; i++) m1 = fmaxf(m1, sc[i][h]);
      const float a = __builtin_amdgcn_exp2f(m[h] - m1);
      l[h] *= a;
#pragma unroll
      for (int c = 0; c < C; c++)
#pragma unroll
        for (int e = 0; e < PER; e++) o[h][c][e] *= a;
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
      const bool own = OWN && owner && cp[i] == pos;
#pragma unroll
      for (int c = 0; c < C; c++) {
        float vf[PER];
        unpack_row<T, PER>(cv[i][c], vf);
#pragma unroll
        for (int e = 0; e < PER; e++) vf[e] = own ? ov[c][e] : vf[e];
#pragma unroll
        for (int h = 0; h < HQ; h++)
#pragma unroll
          for (int e = 0; e < PER; e++) o[h][c][e] = __builtin_fmaf(sc[i][h], vf[e], o[h][c][e]);
      }
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
    for (int c = 0; c < C; c++)
#pragma unroll
      for (int e = 0; e < PER; e += 4) {
        f32x4 v;
#pragma unroll
        for (int k = 0; k < 4; k++) {
          v[k] = o[h][c][e + k] * a;
          if constexpr (GPW > 1) v[k] += __shfl_xor(v[k], 32, 64);
        }
        if (lane < HALF) *reinterpret_cast<f32x4*>(accs + (((w * HQ + h) * C + c) * HALF + lane) * PER + e) = v;
      }
  }
  __syncthreads();
  const size_t rows = (size_t)M * s.heads, r0 = (size_t)sp * rows + (size_t)z * s.heads + h0;
  if (tid < hn) {
    const float lt = (ml[1][0][tid] + ml[1][1][tid]) + (ml[1][2][tid] + ml[1][3][tid]);
    b.part_ml[(r0 + tid) * 2] = fmaxf(fmaxf(ml[0][0][tid], ml[0][1][tid]), fmaxf(ml[0][2][tid], ml[0][3][tid]));
    b.part_ml[(r0 + tid) * 2 + 1] = lt;
  }
  for (uint32_t i = tid; i < hn * s.vdim; i += 256) {
    const uint32_t h = i / s.vdim, d = i % s.vdim, c = d / (LPK * PER), ln = d / PER % LPK, e = d % PER;
    float v = 0.0f;
#pragma unroll
    for (uint32_t k = 0; k < 4; k++)
#pragma unroll
      for (uint32_t x = 0; x < HALF; x += LPK) v += accs[(((k * HQ + h) * C + c) * HALF + x + ln) * PER + e];
    b.part_acc[(r0 + h) * s.vdim + d] = v;
  }
}

template <class T, uint32_t LPK, int HQ, int C, bool OWN>
__global__ void __launch_bounds__(256) gattn_attn_kernel(const GattnShape s, const GattnBufs b, const GlaShape gs, const GlaBufs gb, const int* __restrict__ pos_ptr, uint32_t pos0,
                                                         uint32_t M, uint32_t n_splits, uint32_t n_attn) {
  extern __shared__ __attribute__((aligned(16))) float accs[];      // [4 waves][HQ][C][HALF][PER]
  const uint32_t z = blockIdx.y, pos = (pos_ptr ? (uint32_t)*pos_ptr : pos0) + z;
  if (OWN && blockIdx.x >= n_attn) {
    const uint32_t i = blockIdx.x - n_attn, cols = (gs.vdim + 15) / 16;
    gla_step(gs, gb, pos, i % cols, i / cols);
    return;
  }
  gattn_split<T, LPK, HQ, C, OWN>(s, b, pos, z, M, blockIdx.x % n_splits, blockIdx.x / n_splits, n_splits, accs);
}

static bool gattn_ok(const GattnShape& s) {
  return s.heads && s.kv_heads && s.heads % s.kv_heads == 0 && s.dim && s.dim <= s.dp && s.dp % 64 == 0 && s.dp <= kGattnMaxDim && s.vdim && s.vdim <= s.vp &&
         s.vp % 64 == 0 && s.vp <= kGattnMaxDim && s.chunk && s.window && s.rows % 64 == 0 && s.rot_n <= s.dim && s.rot_n % 2 == 0;
}

template <class T, uint32_t LPK, int HQ, int C>
static hipError_t gattn_attn_go(const GattnShape& s, const GattnBufs& b, const GlaShape* gs, const GlaBufs* gb, const int* pos_ptr, uint32_t pos0, uint32_t M, bool own,
                                uint32_t n_splits, hipStream_t st) {
  const uint32_t gq = s.heads / s.kv_heads, chunks = (gq + HQ - 1) / HQ, n_attn = n_splits * s.kv_heads * chunks;
  const uint32_t n_gla = gs ? gs->heads * ((gs->vdim + 15) / 16) : 0;
  const size_t lds = (size_t)4 * HQ * C * (64 / LPK > 1 ? 32 : 64) * (16 / sizeof(T)) * 4;
  if (own) hipLaunchKernelGGL((gattn_attn_kernel<T, LPK, HQ, C, true>), dim3(n_attn + n_gla, 1), dim3(256), lds, st, s, b, gs ? *gs : GlaShape(), gs ? *gb : GlaBufs(), pos_ptr, pos0, M, n_splits, n_attn);
  else hipLaunchKernelGGL((gattn_attn_kernel<T, LPK, HQ, C, false>), dim3(n_attn, M), dim3(256), lds, st, s, b, GlaShape(), GlaBufs(), pos_ptr, pos0, M, n_splits, n_attn);
  return hipGetLastError();
}
template <class T, uint32_t LPK, int C>
static hipError_t gattn_attn_pick(const GattnShape& s, const GattnBufs& b, const GlaShape* gs, const GlaBufs* gb, const int* pos_ptr, uint32_t pos0, uint32_t M, bool own,
                                  uint32_t n_splits, hipStream_t st) {
  const uint32_t gq = s.heads / s.kv_heads;
  if (gq == 1) return gattn_attn_go<T, LPK, 1, C>(s, b, gs, gb, pos_ptr, pos0, M, own, n_splits, st);
  if (gq == 2 || C == 2) return gattn_attn_go<T, LPK, 2, C>(s, b, gs, gb, pos_ptr, pos0, M, own, n_splits, st);
  if constexpr (C == 1) return gattn_attn_go<T, LPK, 4, C>(s, b, gs, gb, pos_ptr, pos0, M, own, n_splits, st);
  return hipErrorInvalidValue;
}

hipError_t gattn_attn_launch(const GattnShape& s, const GattnBufs& b, const GlaShape* gs, const GlaBufs* gb, const int* pos_ptr, uint32_t pos0, uint32_t M, bool own,
                             uint32_t n_splits, bool f32, hipStream_t st) {
  if (!gattn_ok(s) || M == 0 || M > kGattnShort || (own && M != 1) || (gs && (!gb || !own)) || n_splits == 0 || n_splits > kGattnMaxSplits ||
      (!pos_ptr && pos0 + M > s.rows) || (s.rot_n && !b.cs) || (own && b.shared) || !b.qn != !b.kn)
    return hipErrorInvalidValue;
  const uint32_t bytes = gattn_row_bytes(s, f32);
#define LGH_GATTN_CASE(L, N) \
  return f32 ? gattn_attn_pick<float, L, N>(s, b, gs, gb, pos_ptr, pos0, M, own, n_splits, st) : gattn_attn_pick<__bf16, L, N>(s, b, gs, gb, pos_ptr, pos0, M, own, n_splits, st)
  switch (gattn_lanes(bytes)) {
    case 8: return f32 ? hipErrorInvalidValue : gattn_attn_pick<__bf16, 8, 1>(s, b, gs, gb, pos_ptr, pos0, M, own, n_splits, st);   // (f32 rows have 256 bytes and more)
    case 16: LGH_GATTN_CASE(16, 1);
    case 32: LGH_GATTN_CASE(32, 1);
    case 64:
      if (bytes <= 1024) LGH_GATTN_CASE(64, 1);
      return f32 ? gattn_attn_pick<float, 64, 2>(s, b, gs, gb, pos_ptr, pos0, M, own, n_splits, st) : hipErrorInvalidValue;
  }
#undef LGH_GATTN_CASE
  return hipErrorInvalidValue;
}

// shares of the keys that fill the chip; not more than there are rounds of keys
uint32_t gattn_splits(const GattnShape& s, uint32_t max_seq, uint32_t M, bool f32, uint32_t forced) {
  const uint32_t bytes = gattn_row_bytes(s, f32), gq = s.heads / s.kv_heads, hq = gq <= 2 ? gq : bytes > 1024 ? 2 : 4, wgs = s.kv_heads * ((gq + hq - 1) / hq) * M;
  const uint32_t kr = gattn_round(gattn_lanes(bytes)), rounds = (std::min(std::min(max_seq, s.chunk), s.window) + kr - 1) / kr;
  const uint32_t want = forced ? forced : std::max(1u, 512 / wgs);
  return std::min(std::min(want, kGattnMaxSplits), std::max(rounds, 1u));
}

// ------------------------------------------------------------------------------------------------
// the shares of the keys put together and gated; grid (heads, then heads of the linear attention to read out; tokens).  V: 4 where heads have a
// multiple of 4 values
// ------------------------------------------------------------------------------------------------
template <class O, int V>
__global__ void __launch_bounds__(256) gattn_merge_kernel(const GattnShape s, const GattnBufs b, const GlaShape gs, const GlaBufs gb, uint32_t gla_col,
                                                          const int* __restrict__ pos_ptr, uint32_t pos0, uint32_t M, uint32_t n_splits, uint32_t kr, O* __restrict__ out, uint32_t ldo) {
  struct Val { float v[V]; };
  __shared__ Val part[256];
  __shared__ float wgt[kGattnMaxSplits];
  static_assert(kGattnMaxSplits == 128, "two splits per lane");
  const uint32_t tid = threadIdx.x, lane = tid & 63, h = blockIdx.x, t = blockIdx.y;
  out += (size_t)t * ldo;
  const float* cat = b.cat + (size_t)t * s.ldcat;
  if (h >= s.heads) {
    const uint32_t g = h - s.heads;
    if (tid < 64) gla_read_out<O>(gs, gb.norm, gb.num + (size_t)g * gs.ldo, cat, g, out + gla_col + (size_t)g * gs.vdim);
    return;
  }
  const uint32_t pos = (pos_ptr ? (uint32_t)*pos_ptr : pos0) + t;
  const uint32_t total = pos + 1 - key_start(s, pos), rounds = (total + kr - 1) / kr, per = (rounds + n_splits - 1) / n_splits, act = (rounds + per - 1) / per;
  const size_t rows = (size_t)M * s.heads, r = (size_t)t * s.heads + h;
  // (what the inactive shares hold is not used: the loads need no position)
  f32x2 ml[2];
#pragma unroll
  for (uint32_t k = 0; k < 2; k++) {
    const uint32_t i = lane + k * 64;
    ml[k] = *reinterpret_cast<const f32x2*>(b.part_ml + ((i < n_splits ? i : n_splits - 1) * rows + r) * 2);
  }
  // columns x groups of splits; the first partial sums are requested before the weights are known
  const uint32_t all = (s.vdim + V - 1) / V, cols = all < 256 ? all : 256, groups = 256 / cols, grp = tid / cols;
  auto load = [&](uint32_t k, uint32_t c) {
    Val x;
    const float* p = b.part_acc + (k * rows + r) * s.vdim + c;
    if constexpr (V == 4) { const f32x4 q = *reinterpret_cast<const f32x4*>(p); x.v[0] = q.x; x.v[1] = q.y; x.v[2] = q.z; x.v[3] = q.w; }
    else x.v[0] = p[0];
    return x;
  };
  constexpr int F = 8;
  for (uint32_t base = 0; base < all; base += cols) {   // (one turn unless heads are wide and odd)
    const uint32_t c = base + tid % cols, c0 = (c < all ? c : all - 1) * V;
    Val first[F], v, gt;
#pragma unroll
    for (int i = 0; i < F; i++) first[i] = load(grp + i * groups < n_splits ? grp + i * groups : n_splits - 1, c0);
#pragma unroll
    for (int j = 0; j < V; j++) { gt.v[j] = s.gated ? cat[s.off_g + (size_t)h * s.vdim + c0 + j] : 0.0f; v.v[j] = 0.0f; }
    if (base == 0 && tid < 64) {
      const float m0 = lane < act ? ml[0].x : kGattnNeg, m1 = lane + 64 < act ? ml[1].x : kGattnNeg;
      const float mm = fmaxf(wave_max(fmaxf(m0, m1)), s.sink ? 0.0f : kGattnNeg);
      const float f0 = __builtin_amdgcn_exp2f(m0 - mm), f1 = __builtin_amdgcn_exp2f(m1 - mm);
      const float l0 = lane < act ? f0 * ml[0].y : 0.0f, l1 = lane + 64 < act ? f1 * ml[1].y : 0.0f;
      const float tot = wave_sum(l0 + l1) + (s.sink ? __builtin_amdgcn_exp2f(-mm) : 0.0f);
      wgt[lane] = f0 / tot; wgt[lane + 64] = f1 / tot;
    }
    __syncthreads();
    if (grp < groups) {
#pragma unroll
      for (int i = 0; i < F; i++) {
        const uint32_t k = grp + i * groups;
        if (k < act)
#pragma unroll
          for (int j = 0; j < V; j++) v.v[j] = __builtin_fmaf(wgt[k], first[i].v[j], v.v[j]);
      }
      for (uint32_t k = grp + F * groups; k < act; k += groups) {
        const Val x = load(k, c0);
#pragma unroll
        for (int j = 0; j < V; j++) v.v[j] = __builtin_fmaf(wgt[k], x.v[j], v.v[j]);
      }
    }
    part[tid] = v;
    __syncthreads();
    if (tid < cols && c < all) {
      for (uint32_t k = 1; k < groups; k++)
#pragma unroll
        for (int j = 0; j < V; j++) v.v[j] += part[tid + k * cols].v[j];
#pragma unroll
      for (int j = 0; j < V; j++) out[(size_t)h * s.vdim + c0 + j] = to_act<O>(v.v[j] * (s.gated ? sigmoid_f(gt.v[j]) : 1.0f) * s.out_scale);
    }
    __syncthreads();
  }
}

hipError_t gattn_merge_launch(const GattnShape& s, const GattnBufs& b, const GlaShape* gs, const GlaBufs* gb, uint32_t gla_col, const int* pos_ptr, uint32_t pos0, uint32_t M,
                              uint32_t n_splits, bool f32, void* out, uint32_t ldo, bool out_f32, hipStream_t st) {
  if (!gattn_ok(s) || n_splits == 0 || n_splits > kGattnMaxSplits || M == 0 || (gs && (!gb || M != 1))) return hipErrorInvalidValue;
  const uint32_t kr = gattn_round(gattn_lanes(gattn_row_bytes(s, f32)));
  const dim3 grid(s.heads + (gs ? gs->heads : 0), M);
  const GlaShape g = gs ? *gs : GlaShape();
  const GlaBufs h = gs ? *gb : GlaBufs();
  const bool v4 = s.vdim % 4 == 0;
#define LGH_MERGE(O, V) hipLaunchKernelGGL((gattn_merge_kernel<O, V>), grid, dim3(256), 0, st, s, b, g, h, gla_col, pos_ptr, pos0, M, n_splits, kr, (O*)out, ldo)
  if (out_f32 && v4) LGH_MERGE(float, 4);
  else if (out_f32) LGH_MERGE(float, 1);
  else if (v4) LGH_MERGE(__bf16, 4);
  else LGH_MERGE(__bf16, 1);
#undef LGH_MERGE
  return hipGetLastError();
}

// ------------------------------------------------------------------------------------------------
// a block's cache rows and queries; grid (tokens, groups of kPrepHeads heads), a wave per head
// ------------------------------------------------------------------------------------------------
constexpr uint32_t kPrepHeads = 8;

template <class T>
__global__ void __launch_bounds__(256) gattn_prep_kernel(const GattnShape s, const GattnBufs b, uint32_t pos0) {
  const uint32_t t = blockIdx.x, pos = pos0 + t, lane = threadIdx.x & 63, w = (uint32_t)__builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6));
  const float* cat = b.cat + (size_t)t * s.ldcat;
  const f32x2* cs = reinterpret_cast<const f32x2*>(b.cs) + (size_t)pos * (s.rot_n / 2);
  constexpr uint32_t NP = kGattnMaxDim / 128;                       // pairs of a lane
  auto store2 = [](T* p, float u, float v) {
    T o[2] = {to_act<T>(u), to_act<T>(v)};
    __builtin_memcpy(__builtin_assume_aligned(p, sizeof(o)), o, sizeof(o));
  };
  const uint32_t nh = s.heads + (b.shared ? 0 : s.kv_heads);
  const bool normed = b.qn != nullptr;
  const uint32_t i0 = (b.q ? 0 : s.heads) + blockIdx.y * kPrepHeads, i1 = i0 + kPrepHeads < nh ? i0 + kPrepHeads : nh;
  for (uint32_t i = i0 + w; i < i1; i += 4) {
    const bool key = i >= s.heads;
    const uint32_t h = key ? i - s.heads : i;
    const float* p = cat + (key ? s.off_k : s.off_q) + (size_t)h * s.dim;
    const float* nw = key ? b.kn : b.qn;
    f32x2 x[NP], n[NP], r[NP];
    float ss = 0.0f;
#pragma unroll
    for (uint32_t j = 0; j < NP; j++) {
      const uint32_t d = j * 128 + lane * 2;
      x[j] = (f32x2)(0.0f);
      n[j] = (f32x2)(1.0f);
      r[j].x = 1.0f; r[j].y = 0.0f;
      if (j * 128 < s.dim) {
        if (d < s.dim) { x[j].x = p[d]; if (normed) n[j].x = nw[d]; }
        if (d + 1 < s.dim) { x[j].y = p[d + 1]; if (normed) n[j].y = nw[d + 1]; }
        if (d + 1 < s.rot_n) r[j] = cs[d / 2];
      }
      ss = __builtin_fmaf(x[j].x, x[j].x, __builtin_fmaf(x[j].y, x[j].y, ss));
    }
    const float inv = normed ? 1.0f / __builtin_sqrtf(wave_sum(ss) / (float)s.dim + s.eps) : 1.0f, f = key ? 1.0f : s.scale * kGattnLog2e;
    T* o = key ? reinterpret_cast<T*>(b.kc) + ((size_t)h * s.rows + pos) * s.dp : reinterpret_cast<T*>(b.q) + ((size_t)h * b.Mcap + t) * s.dp;
#pragma unroll
    for (uint32_t j = 0; j < NP; j++) {
      const uint32_t d = j * 128 + lane * 2;
      const f32x2 v = rotate2(x[j].x * inv * n[j].x, x[j].y * inv * n[j].y, r[j]);
      if (d < s.dp) store2(o + d, v.x * f, v.y * f);
    }
  }
  if (b.shared) return;
  for (uint32_t i = blockIdx.y * 256 + threadIdx.x; i < s.kv_heads * s.vdim; i += 256 * gridDim.y)
    reinterpret_cast<T*>(b.vc)[((size_t)(i / s.vdim) * s.rows + pos) * s.vp + i % s.vdim] = to_act<T>(cat[s.off_v + i]);
}

hipError_t gattn_prep_launch(const GattnShape& s, const GattnBufs& b, uint32_t pos0, uint32_t M, bool f32, hipStream_t st) {
  if (!gattn_ok(s) || M == 0 || (b.q && M > b.Mcap) || pos0 + M > s.rows || (s.rot_n && !b.cs) || !b.qn != !b.kn) return hipErrorInvalidValue;
  if (b.shared && !b.q) return hipSuccess;
  const dim3 grid(M, ((b.q ? s.heads : 0) + (b.shared ? 0 : s.kv_heads) + kPrepHeads - 1) / kPrepHeads);
  if (f32) hipLaunchKernelGGL((gattn_prep_kernel<float>), grid, dim3(256), 0, st, s, b, pos0);
  else hipLaunchKernelGGL((gattn_prep_kernel<__bf16>), grid, dim3(256), 0, st, s, b, pos0);
  return hipGetLastError();
}

// ------------------------------------------------------------------------------------------------
// prompt portions.  A workgroup = 4 waves = 64 * QT queries of one head (and DV of its values); S^T = K Q^T leaves a lane with one query's scores of
// keys 4g .. 4g + 3, which is the operand of O^T = V^T P^T, whose value fragments come out of LDS by transposed reads.  Tiles of KT keys and values
// go to LDS by DMA, two buffers.
// ------------------------------------------------------------------------------------------------
template <class T> constexpr int gattn_kt() { return sizeof(T) == 2 ? 64 : 32; }
template <class T, int DQ, int DV> constexpr size_t gattn_lds() { return 2 * (size_t)gattn_kt<T>() * (DQ + DV) * sizeof(T); }
template <class T, int DQ, int DV> constexpr int gattn_qt() { return sizeof(T) == 2 && DQ + DV <= 384 ? 2 : 1; }   // 16-query tiles per wave
template <class T, int DQ, int DV> constexpr int gattn_wgs() { return gattn_lds<T, DQ, DV>() <= 80 * 1024 && DQ + DV <= 256 ? 2 : 1; }

template <class T, int DQ, int DV>
__global__ void __launch_bounds__(256, (gattn_wgs<T, DQ, DV>())) gattn_flash_kernel(const GattnShape s, const GattnBufs b, uint32_t pos0, uint32_t M, uint32_t nqb, T* __restrict__ out,
                                                                                    uint32_t ldo) {
  constexpr bool BF = sizeof(T) == 2;
  constexpr int KT = gattn_kt<T>(), QT = gattn_qt<T, DQ, DV>(), NK = KT / 16, NU = DQ / Frag<T>::KU, ND = DV / 16;
  constexpr uint32_t XK = DQ * sizeof(T) / 16, XV = DV * sizeof(T) / 16, kKBytes = KT * XK * 16, kVBytes = KT * XV * 16, kBuf = kKBytes + kVBytes;
  extern __shared__ __attribute__((aligned(16))) uint8_t smem[];
  const uint32_t lane = threadIdx.x & 63, w = (uint32_t)__builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6)), r16 = lane & 15, g = lane >> 4;
  // the longest rows first, and of the second half of the grid the shortest first (workgroups i and i + half share a CU when all are resident)
  const uint32_t h = blockIdx.x % s.heads, qi = blockIdx.x / s.heads, hi = (nqb + 1) / 2, qb = qi < hi ? nqb - 1 - qi : qi - hi, v0 = blockIdx.y * DV;
  const uint32_t q0 = qb * 64 * QT, qw = q0 + w * 16 * QT, qlast = q0 + 64 * QT - 1 < M - 1 ? q0 + 64 * QT - 1 : M - 1;
  const uint32_t tw = key_start(s, pos0 + q0) / KT, tiles = (pos0 + qlast) / KT + 1 - tw;
  const uint32_t kh = h / (s.heads / s.kv_heads);
  const T* K = reinterpret_cast<const T*>(b.kc) + (size_t)kh * s.rows * DQ;
  const T* Vc = reinterpret_cast<const T*>(b.vc) + (size_t)kh * s.rows * s.vp + v0;
  const uint32_t lds0 = (uint32_t)__builtin_amdgcn_readfirstlane((int)lds_addr_of(smem));
  auto stage = [&](uint32_t tl, uint32_t buf) {
#pragma unroll
    for (int i = 0; i < (int)(kKBytes / 4096); i++) {
      const uint32_t c = (i * 4 + w) * 64 + lane, row = c / XK, ch = (c % XK) ^ (row & 7);
      lds_dma16_untracked(K + ((size_t)tl * KT + row) * DQ + ch * (16 / sizeof(T)), lds0 + buf * kBuf + (i * 4 + w) * 1024);
    }
#pragma unroll
    for (int i = 0; i < (int)(kVBytes / 4096); i++) {
      const uint32_t c = (i * 4 + w) * 64 + lane, row = c / XV, ch = (c % XV) ^ (row & 7);
      lds_dma16_untracked(Vc + ((size_t)tl * KT + row) * s.vp + ch * (16 / sizeof(T)), lds0 + buf * kBuf + kKBytes + (i * 4 + w) * 1024);
    }
  };
  stage(tw, 0);
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
  uint32_t ci[QT];                                              // the first key that this lane's query sees
#pragma unroll
  for (int t = 0; t < QT; t++) {
    mx[t] = s.sink ? 0.0f : kGattnNeg;                          // the sink: a first key of score 0 and no value
    l[t] = s.sink && g == 0 ? 1.0f : 0.0f;
    ci[t] = key_start(s, pos0 + qw + t * 16 + r16);
#pragma unroll
    for (int i = 0; i < ND; i++) o[i][t] = (f32x4)(0.0f);
  }
  const uint32_t iw0 = pos0 + qw, iw1 = iw0 + 16 * QT - 1;      // this wave's queries
  const uint32_t c0 = key_start(s, iw0), c1 = key_start(s, iw1);
  wait_vm(0);
  __syncthreads();
  for (uint32_t it = 0; it < tiles; it++) {
    const uint32_t cur = it & 1, k0 = (tw + it) * KT, k1 = k0 + KT - 1;
    if (it + 1 < tiles) stage(tw + it + 1, cur ^ 1);
    // (wave-uniform) no query of this wave sees the tile / every one sees all of it
    const bool none = k0 > iw1 || k1 < c0, full = k1 <= iw0 && k0 >= c1;
    if (!none) {
      const T* tile = reinterpret_cast<const T*>(smem + cur * kBuf);
      const T* vtile = reinterpret_cast<const T*>(smem + cur * kBuf + kKBytes);
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
#pragma unroll
      for (int t = 0; t < QT; t++) {
        if (!full) {
          asm volatile("");              // (kept a branch: most tiles have no masks to apply)
          const uint32_t i = iw0 + t * 16 + r16;
#pragma unroll
          for (int n = 0; n < NK; n++)
#pragma unroll
            for (int e = 0; e < 4; e++) {
              const uint32_t j = k0 + n * 16 + g * 4 + e;
              sa[n][t][e] = j <= i && j >= ci[t] ? sa[n][t][e] : kGattnNeg;
            }
        }
        float m1 = kGattnNeg;
#pragma unroll
        for (int n = 0; n < NK; n++)
#pragma unroll
          for (int e = 0; e < 4; e++) m1 = fmaxf(m1, sa[n][t][e]);
        m1 = fmaxf(m1, __shfl_xor(m1, 16, 64));
        m1 = fmaxf(m1, __shfl_xor(m1, 32, 64));
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
        float sum = 0.0f;
#pragma unroll
        for (int n = 0; n < NK; n++)
#pragma unroll
          for (int e = 0; e < 4; e++) {
            const float p = __builtin_amdgcn_exp2f(sa[n][t][e] - mx[t]);
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
            const bf16x8 vf = tile_value_frag<T>(vtile + u * 32 * DV, DV, 0, d * 16, r16, g);
#pragma unroll
            for (int t = 0; t < QT; t++) o[d][t] = Frag<T>::mma(vf, pf[t], o[d][t]);
          }
        }
      } else {
#pragma unroll
        for (int n = 0; n < NK; n++)
#pragma unroll
          for (int d = 0; d < ND; d++) {
            const f32x4 vf = tile_value_frag<T>(vtile, DV, n, d * 16, r16, g);
#pragma unroll
            for (int t = 0; t < QT; t++) o[d][t] = Frag<T>::mma(vf, sa[n][t], o[d][t]);
          }
      }
      __builtin_amdgcn_s_setprio(0);
    }
    wait_vm(0);
    __syncthreads();
  }
#pragma unroll
  for (int t = 0; t < QT; t++) {
    float lt = l[t];
    lt += __shfl_xor(lt, 16, 64);
    lt += __shfl_xor(lt, 32, 64);
    const uint32_t m = qw + t * 16 + r16;
    if (m >= M) continue;
    const float fac = s.out_scale / lt;
    const float* gt = b.cat + (size_t)m * s.ldcat + s.off_g + (size_t)h * s.vdim;
    T* dst = out + (size_t)m * ldo + (size_t)h * s.vdim;
    const bool vec = (s.vdim & 3) == 0;
#pragma unroll
    for (int d = 0; d < ND; d++) {
      const uint32_t v = v0 + d * 16 + g * 4;
      if (v >= s.vdim) continue;
      if (vec) {
        f32x4 z = (f32x4)(0.0f);
        if (s.gated) z = *reinterpret_cast<const f32x4*>(gt + v);
        T r[4];
#pragma unroll
        for (int e = 0; e < 4; e++) r[e] = to_act<T>(o[d][t][e] * fac * (s.gated ? sigmoid_f(z[e]) : 1.0f));
        __builtin_memcpy(__builtin_assume_aligned(dst + v, sizeof(r)), r, sizeof(r));
      } else {
#pragma unroll
        for (int e = 0; e < 4; e++)
          if (v + e < s.vdim) dst[v + e] = to_act<T>(o[d][t][e] * fac * (s.gated ? sigmoid_f(gt[v + e]) : 1.0f));
      }
    }
  }
}

template <class T, int DQ, int DV>
static hipError_t gattn_flash_go(const GattnShape& s, const GattnBufs& b, uint32_t pos0, uint32_t M, void* out, uint32_t ldo, hipStream_t st) {
  static bool opted[64] = {};
  constexpr size_t lds = gattn_lds<T, DQ, DV>();
  static_assert(lds <= 160 * 1024, "two tiles of keys and values fit LDS");
  if (hipError_t e = lds_opt_in(reinterpret_cast<const void*>(&gattn_flash_kernel<T, DQ, DV>), (int)lds, opted); e != hipSuccess) return e;
  const uint32_t QB = 64 * gattn_qt<T, DQ, DV>(), nqb = (M + QB - 1) / QB;
  hipLaunchKernelGGL((gattn_flash_kernel<T, DQ, DV>), dim3(nqb * s.heads, s.vp / DV), dim3(256), lds, st, s, b, pos0, M, nqb, (T*)out, ldo);
  return hipGetLastError();
}
template <class T, int DQ>
static hipError_t gattn_flash_pick(const GattnShape& s, const GattnBufs& b, uint32_t pos0, uint32_t M, void* out, uint32_t ldo, hipStream_t st) {
  switch (s.vp) {
    case 64: return gattn_flash_go<T, DQ, 64>(s, b, pos0, M, out, ldo, st);
    case 128: return gattn_flash_go<T, DQ, 128>(s, b, pos0, M, out, ldo, st);
    case 192: return gattn_flash_go<T, DQ, 192>(s, b, pos0, M, out, ldo, st);
    case 256: case 512: return gattn_flash_go<T, DQ, 256>(s, b, pos0, M, out, ldo, st);
    case 320: return gattn_flash_go<T, DQ, 64>(s, b, pos0, M, out, ldo, st);
    case 384: return gattn_flash_go<T, DQ, 192>(s, b, pos0, M, out, ldo, st);
    case 448: return gattn_flash_go<T, DQ, 64>(s, b, pos0, M, out, ldo, st);
  }
  return hipErrorInvalidValue;
}

hipError_t gattn_flash_launch(const GattnShape& s, const GattnBufs& b, uint32_t pos0, uint32_t M, bool f32, void* out, uint32_t ldo, hipStream_t st) {
  // whole tiles of keys and values are read
  if (!gattn_ok(s) || !b.q || M == 0 || M > b.Mcap || (uint64_t)(pos0 + M + 63) / 64 * 64 > s.rows || ldo < s.heads * s.vdim || (ldo & 3)) return hipErrorInvalidValue;
#define LGH_FLASH_CASE(Q) case Q: return f32 ? gattn_flash_pick<float, Q>(s, b, pos0, M, out, ldo, st) : gattn_flash_pick<__bf16, Q>(s, b, pos0, M, out, ldo, st)
  switch (s.dp) {
    LGH_FLASH_CASE(64); LGH_FLASH_CASE(128); LGH_FLASH_CASE(192); LGH_FLASH_CASE(256);
  }
#undef LGH_FLASH_CASE
  return hipErrorInvalidValue;
}

}  // namespace lgh
