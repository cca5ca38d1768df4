// delta.hip — the gated delta rule of layered.h, all of it in 32-bit (running sums of log decays in 64-bit).  Queries, keys and values pass a short
// causal convolution and silu; queries and keys are unit vectors.  Per head, with log decay l_t = -exp(A_log) softplus(a_t + dt) and step beta_t:
//   u_t = beta_t (v_t - exp(l_t) S_(t-1)^T k_t),   S_t = exp(l_t) S_(t-1) + k_t u_t^T,   o_t = S_t^T q_t.
//
// A block goes 64 tokens at a time.  With b_t the sum of l up to t within the chunk (b_e at its end) and S_p the state before it, the u_t solve
//   (I + L) U = B V - B E K S_p,   L_ts = beta_t exp(b_t - b_s) k_t . k_s (s < t),   B = diag(beta), E = diag(exp(b)),
// so U = U0 - W S_p with U0 = (I + L)^-1 B V and W = (I + L)^-1 B E K, and with A_ts = exp(b_t - b_s) q_t . k_s (s <= t)
//   O = E Q S_p + A U = P S_p + A U0,   P = E Q - A W,      S_e = exp(b_e) S_p + sum_s exp(b_e - b_s) k_s u_s^T.
// Everything but the two products with S_p and the state's update is free of the recurrence: U0, W, P and A U0 are formed for all chunks at once.  No
// exponent is positive.  (I + L) is solved 16 tokens at a time: the four diagonal blocks are inverted by substitution, the rest are products on the f32
// matrix cores, whose result tiles are operands of the next product as they lie in the registers.
#include "layered.h"
#include "layered_device.h"

namespace lgh {

__device__ __forceinline__ float delta_log_decay(float a_log, float dt, float a) { return -expf(a_log) * softplus_f(a + dt); }
__device__ __forceinline__ float silu_hw(float z) { return z * sigmoid_hw(z); }

// a wave-uniform place (in floats) and this lane's distance from it (in bytes): one address register for all the rows that a lane touches
__device__ __forceinline__ float at1(const float* base, size_t row, uint32_t lane_off) { return *reinterpret_cast<const float*>(reinterpret_cast<const char*>(base + row) + lane_off); }
__device__ __forceinline__ f32x4 at4(const float* base, size_t row, uint32_t lane_off) { return *reinterpret_cast<const f32x4*>(reinterpret_cast<const char*>(base + row) + lane_off); }
__device__ __forceinline__ void put1(float* base, size_t row, uint32_t lane_off, float v) { *reinterpret_cast<float*>(reinterpret_cast<char*>(base + row) + lane_off) = v; }

// the convolution's output of channel c at position pos, x: its input there
__device__ __forceinline__ float delta_conv_step(const DeltaShape& s, const DeltaBufs& b, uint32_t pos, uint32_t c, float x) {
  const float* w = b.conv + (size_t)c * s.taps;
  float v = w[s.taps - 1] * x;
  uint32_t r = pos % s.taps;
  for (uint32_t j = 1; j < s.taps; j++) {
    r = r ? r - 1 : s.taps - 1;
    const float h = b.hist[(size_t)r * s.cols + c];
    v = __builtin_fmaf(w[s.taps - 1 - j], j <= pos ? h : 0.0f, v);
  }
  return silu_hw(v);
}

// ------------------------------------------------------------------------------------------------
// decode: one token.  A workgroup owns 16 columns of one head's state (4 lanes x 4 columns, 64 rows at a time).  S is read once: with the decayed
// state D, u = beta (v - D^T k) and o = D^T q + (k . q) u.  NT: groups of 64 rows held in registers (BIG: the rest is read again for the update)
// ------------------------------------------------------------------------------------------------
template <int NT, bool BIG>
__global__ void __launch_bounds__(256) delta_step_kernel(const DeltaShape s, const DeltaBufs b, const int* __restrict__ pos_ptr, uint32_t pos0) {
  extern __shared__ __attribute__((aligned(16))) float qk[];        // queries, keys [rows]
  __shared__ float vs[16], sums[3][4], o_s[4][2][16];
  const uint32_t h = blockIdx.y, hk = h / (s.heads / s.kv_heads), tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, cq = (tid & 3) * 4, r0 = tid >> 2;
  const uint32_t pos = pos_ptr ? (uint32_t)*pos_ptr : pos0, rows = (s.dk + NT * 64 - 1) / (NT * 64) * (NT * 64);
  const bool lead = blockIdx.x == 0 && h % (s.heads / s.kv_heads) == 0;
  float* S = b.S + (size_t)h * s.dk * s.lv + blockIdx.x * 16 + cq;
  f32x4 st[NT];
  auto fetch = [&](uint32_t d0) {
#pragma unroll
    for (int i = 0; i < NT; i++) {
      const uint32_t d = d0 + i * 64 + r0;
      st[i] = *reinterpret_cast<const f32x4*>(S + (size_t)(d < s.dk ? d : s.dk - 1) * s.lv);
    }
  };
  fetch(0);
  const float zb = b.cat[s.off_b + h], la = delta_log_decay(b.a_log[h], b.dt[h], b.cat[s.off_a + h]);
  const uint32_t ring = pos % s.taps;
  float ssq = 0.0f, ssk = 0.0f, sqk = 0.0f;
  for (uint32_t i = tid; i < rows; i += 256) {
    float q = 0.0f, k = 0.0f;
    if (i < s.dim) {
      const uint32_t c0 = s.off_q + hk * s.dim + i, c1 = s.off_k + hk * s.dim + i;
      const float xq = b.cat[c0], xk = b.cat[c1];
      q = delta_conv_step(s, b, pos, c0, xq);
      k = delta_conv_step(s, b, pos, c1, xk);
      if (lead) { b.hist[(size_t)ring * s.cols + c0] = xq; b.hist[(size_t)ring * s.cols + c1] = xk; }
    }
    qk[i] = q;
    qk[rows + i] = k;
    ssq = __builtin_fmaf(q, q, ssq); ssk = __builtin_fmaf(k, k, ssk); sqk = __builtin_fmaf(q, k, sqk);
  }
  if (tid >= 192 && tid < 208) {                                    // (a wave without rows where heads are small)
    const uint32_t c = blockIdx.x * 16 + tid - 192, ch = s.off_v + h * s.vdim + c;
    float v = 0.0f;
    if (c < s.vdim) {
      const float x = b.cat[ch];
      v = delta_conv_step(s, b, pos, ch, x);
      b.hist[(size_t)ring * s.cols + ch] = x;
    }
    vs[tid - 192] = v;
  }
  ssq = wave_total(ssq); ssk = wave_total(ssk); sqk = wave_total(sqk);
  if (lane == 0) { sums[0][wv] = ssq; sums[1][wv] = ssk; sums[2][wv] = sqk; }
  __syncthreads();
  auto tot = [&](int i) { return (sums[i][0] + sums[i][1]) + (sums[i][2] + sums[i][3]); };
  const float iq = 1.0f / (__builtin_sqrtf(tot(0) + 1e-6f) * __builtin_sqrtf((float)s.dim)), ik = 1.0f / __builtin_sqrtf(tot(1) + 1e-6f);
  const float kq = tot(2) * iq * ik, g = pos ? expf(la) : 0.0f, beta = sigmoid_f(zb);
  float a[4] = {0.0f, 0.0f, 0.0f, 0.0f}, c[4] = {0.0f, 0.0f, 0.0f, 0.0f};
  for (uint32_t d0 = 0; d0 < rows; d0 += NT * 64) {
    if (BIG && d0) fetch(d0);
#pragma unroll
    for (int i = 0; i < NT; i++) {
      const float qd = qk[d0 + i * 64 + r0], kd = qk[rows + d0 + i * 64 + r0];
#pragma unroll
      for (int e = 0; e < 4; e++) {
        const float x = pos ? st[i][e] : 0.0f;                       // at position 0 whatever is stored belongs to another sequence
        if (!BIG) st[i][e] = x;
        a[e] = __builtin_fmaf(x, kd, a[e]);
        c[e] = __builtin_fmaf(x, qd, c[e]);
      }
    }
  }
#pragma unroll
  for (int e = 0; e < 4; e++) {                                     // the 16 row slots of a wave: lanes with equal lane & 3
    a[e] += __shfl_xor(a[e], 4, 64); a[e] += __shfl_xor(a[e], 8, 64); a[e] += __shfl_xor(a[e], 16, 64); a[e] += __shfl_xor(a[e], 32, 64);
    c[e] += __shfl_xor(c[e], 4, 64); c[e] += __shfl_xor(c[e], 8, 64); c[e] += __shfl_xor(c[e], 16, 64); c[e] += __shfl_xor(c[e], 32, 64);
    if (lane < 4) { o_s[wv][0][lane * 4 + e] = a[e]; o_s[wv][1][lane * 4 + e] = c[e]; }
  }
  __syncthreads();
  auto col = [&](int i, uint32_t x) { return (o_s[0][i][x] + o_s[1][i][x]) + (o_s[2][i][x] + o_s[3][i][x]); };
  auto write = [&](uint32_t x) { return beta * (vs[x] - g * ik * col(0, x)); };   // u of column x
  float u[4];
#pragma unroll
  for (int e = 0; e < 4; e++) u[e] = write(cq + e) * ik;             // (keys lie unscaled in LDS)
  for (uint32_t d0 = 0; d0 < rows; d0 += NT * 64) {
    if (BIG) fetch(d0);
#pragma unroll
    for (int i = 0; i < NT; i++) {
      const uint32_t d = d0 + i * 64 + r0;
      if (d >= s.dk) continue;
      const float kd = qk[rows + d];
      f32x4 x;
#pragma unroll
      for (int e = 0; e < 4; e++) x[e] = __builtin_fmaf(kd, u[e], pos ? g * st[i][e] : 0.0f);
      *reinterpret_cast<f32x4*>(S + (size_t)d * s.lv) = x;
    }
  }
  if (tid < 16) b.num[(size_t)h * s.lv + blockIdx.x * 16 + tid] = __builtin_fmaf(kq, write(tid), g * iq * col(1, tid));
}

static bool delta_ok(const DeltaShape& s) {
  return s.heads && s.kv_heads && s.heads % s.kv_heads == 0 && s.dim && s.vdim && s.taps && s.dk % 16 == 0 && s.dk >= s.dim && s.lv % 16 == 0 && s.lv >= s.vdim &&
         s.off_q + s.kv_heads * s.dim <= s.cols && s.off_k + s.kv_heads * s.dim <= s.cols && s.off_v + s.heads * s.vdim <= s.cols && s.cols <= s.ldcat;
}

template <int NT, bool BIG>
static hipError_t delta_step_go(const DeltaShape& s, const DeltaBufs& b, const int* pos_ptr, uint32_t pos0, hipStream_t st) {
  static bool opted[64] = {};
  const size_t lds = (size_t)(s.dk + NT * 64 - 1) / (NT * 64) * (NT * 64) * 8;
  if (lds > 150 * 1024) return hipErrorInvalidValue;
  if (hipError_t e = lds_opt_in(reinterpret_cast<const void*>(&delta_step_kernel<NT, BIG>), 150 * 1024, opted); e != hipSuccess) return e;
  hipLaunchKernelGGL((delta_step_kernel<NT, BIG>), dim3(s.lv / 16, s.heads), dim3(256), lds, st, s, b, pos_ptr, pos0);
  return hipGetLastError();
}

hipError_t delta_step_launch(const DeltaShape& s, const DeltaBufs& b, const int* pos_ptr, uint32_t pos0, hipStream_t st) {
  if (!delta_ok(s)) return hipErrorInvalidValue;
  if (s.dk <= 64) return delta_step_go<1, false>(s, b, pos_ptr, pos0, st);
  if (s.dk <= 128) return delta_step_go<2, false>(s, b, pos_ptr, pos0, st);
  if (s.dk <= 256) return delta_step_go<4, false>(s, b, pos_ptr, pos0, st);
  return delta_step_go<4, true>(s, b, pos_ptr, pos0, st);
}

// ------------------------------------------------------------------------------------------------
// blocks: convolution, silu, unit vectors.  A wave = 8 tokens of one head (queries, keys, values), 64 * NC channels at a time; grid (32 tokens, heads)
// ------------------------------------------------------------------------------------------------
constexpr int kDeltaTok = 8;

template <int NC>
__global__ void __launch_bounds__(256) delta_prep_kernel(const DeltaShape s, const DeltaBufs b, uint32_t pos0, uint32_t M) {
  const uint32_t lane = threadIdx.x & 63, w = (uint32_t)__builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6)), G = s.kv_heads;
  const uint32_t hh = blockIdx.y, kind = hh < G ? 0 : hh < 2 * G ? 1 : 2, h = hh - (kind == 0 ? 0 : kind == 1 ? G : 2 * G);
  const uint32_t size = kind == 2 ? s.vdim : s.dim, pad = kind == 2 ? s.lv : s.dk, off = (kind == 0 ? s.off_q : kind == 1 ? s.off_k : s.off_v) + h * size;
  float* out = (kind == 0 ? b.q : kind == 1 ? b.k : b.v) + (size_t)h * pad;
  const size_t ld = (size_t)(kind == 2 ? s.heads : G) * pad;
  const int t0 = (int)((blockIdx.x * 4 + w) * kDeltaTok);
  auto input = [&](int t, uint32_t c) -> float {                    // (t may lie before the block)
    if (t >= 0) return b.cat[(size_t)(t < (int)M ? t : (int)M - 1) * s.ldcat + c];
    const int p = (int)pos0 + t;
    return p >= 0 ? b.hist[(size_t)((uint32_t)p % s.taps) * s.cols + c] : 0.0f;
  };
  for (uint32_t c0 = 0; c0 < pad; c0 += 64 * NC) {                  // (one turn for queries and keys)
    float x[NC][kDeltaTok];
#pragma unroll
    for (int n = 0; n < NC; n++) {
      const uint32_t c = c0 + n * 64 + lane, ch = off + (c < size ? c : size - 1);
      const float* f = b.conv + (size_t)ch * s.taps;
      if (s.taps <= 4) {                                            // a window of inputs in registers
        float in[kDeltaTok + 3], fl[4];
#pragma unroll
        for (int i = 0; i < 4; i++) fl[i] = i < (int)s.taps ? f[s.taps - 1 - i] : 0.0f;   // fl[i]: i positions back
        if (t0 > 0 && t0 + kDeltaTok <= (int)M) {
          const float* p = b.cat + (size_t)(t0 - 3) * s.ldcat + ch;
#pragma unroll
          for (int i = 0; i < kDeltaTok + 3; i++) in[i] = p[(size_t)i * s.ldcat];
        } else {
#pragma unroll
          for (int i = 0; i < kDeltaTok + 3; i++) in[i] = i >= 3 || (int)s.taps > 3 - i ? input(t0 + i - 3, ch) : 0.0f;
        }
#pragma unroll
        for (int i = 0; i < kDeltaTok; i++) x[n][i] = __builtin_fmaf(fl[0], in[i + 3], __builtin_fmaf(fl[1], in[i + 2], __builtin_fmaf(fl[2], in[i + 1], fl[3] * in[i])));
      } else {
#pragma unroll
        for (int i = 0; i < kDeltaTok; i++) x[n][i] = 0.0f;
        for (uint32_t j = 0; j < s.taps; j++) {
          const float fj = f[s.taps - 1 - j];
#pragma unroll
          for (int i = 0; i < kDeltaTok; i++) x[n][i] = __builtin_fmaf(fj, input(t0 + i - (int)j, ch), x[n][i]);
        }
      }
#pragma unroll
      for (int i = 0; i < kDeltaTok; i++) x[n][i] = c < size && t0 + i < (int)M ? silu_hw(x[n][i]) : 0.0f;
    }
#pragma unroll
    for (int i = 0; i < kDeltaTok; i++) {
      float f = 1.0f;
      if (kind != 2) {
        float ss = 0.0f;
#pragma unroll
        for (int n = 0; n < NC; n++) ss = __builtin_fmaf(x[n][i], x[n][i], ss);
        f = 1.0f / __builtin_sqrtf(wave_total(ss) + 1e-6f);
        if (kind == 0) f /= __builtin_sqrtf((float)s.dim);
      }
#pragma unroll
      for (int n = 0; n < NC; n++) {
        const uint32_t c = c0 + n * 64 + lane;
        if (c < pad) out[(size_t)(t0 + i) * ld + c] = x[n][i] * f;
      }
    }
  }
}

// ------------------------------------------------------------------------------------------------
// blocks: what a chunk is without the state before it; grid (chunks, heads)
// ------------------------------------------------------------------------------------------------
constexpr uint32_t kScLd = 68, kTiLd = 20;

__global__ void __launch_bounds__(256) delta_chunk_kernel(const DeltaShape s, const DeltaBufs b, uint32_t M) {
  __shared__ __attribute__((aligned(16))) float L[64][kScLd], A[64][kScLd], T[4][16][kTiLd];
  __shared__ double bs[64];
  __shared__ __attribute__((aligned(16))) float bet[64], eb[64];
  const uint32_t ch = blockIdx.x, h = blockIdx.y, G = s.kv_heads, hk = h / (s.heads / G), t0 = ch * 64;
  const uint32_t lane = threadIdx.x & 63, w = (uint32_t)__builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6)), r16 = lane & 15, g = lane >> 4;
  const float* K = b.k + ((size_t)t0 * G + hk) * s.dk;
  const float* Q = b.q + ((size_t)t0 * G + hk) * s.dk;
  const size_t ldk = (size_t)G * s.dk, ldw = (size_t)s.heads * s.dk, ldv = (size_t)s.heads * s.lv;
  if (w == 0) {
    const uint32_t t = t0 + lane;
    const float* row = b.cat + (size_t)(t < M ? t : M - 1) * s.ldcat;
    const float la = delta_log_decay(b.a_log[h], b.dt[h], row[s.off_a + h]), be = sigmoid_f(row[s.off_b + h]);
    double r = t < M ? (double)la : 0.0;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) { const double p = __shfl_up(r, o, 64); if ((int)lane >= o) r += p; }
    const double re = __shfl(r, 63, 64);
    bs[lane] = r;
    bet[lane] = t < M ? be : 0.0f;
    eb[lane] = expf((float)r);
    b.wge[(size_t)h * b.Mcap + t] = expf((float)(re - r));
    if (lane == 0) b.cd[(size_t)h * (b.Mcap / 64) + ch] = expf((float)re);
  }
  // scores of wave w's 16 tokens with the keys up to them
  f32x4 kk[4], qq[4];
#pragma unroll
  for (int j = 0; j < 4; j++) { kk[j] = (f32x4)(0.0f); qq[j] = (f32x4)(0.0f); }
  {
    const uint32_t lo = (r16 * (uint32_t)ldk + g * 4) * 4;
    for (uint32_t d = 0; d < s.dk; d += 16) {
      const f32x4 kf = at4(K, w * 16 * ldk + d, lo), qf = at4(Q, w * 16 * ldk + d, lo);
#pragma unroll
      for (int j = 0; j < 4; j++) {
        if (j > (int)w) continue;                                    // (wave-uniform)
        const f32x4 xf = at4(K, j * 16 * ldk + d, lo);
        kk[j] = Frag<float>::mma(kf, xf, kk[j]);
        qq[j] = Frag<float>::mma(qf, xf, qq[j]);
      }
    }
  }
  __syncthreads();
#pragma unroll
  for (int j = 0; j < 4; j++) {
    if (j > (int)w) continue;
    const uint32_t sc = j * 16 + r16;
    const double bk = bs[sc];
#pragma unroll
    for (int e = 0; e < 4; e++) {
      const uint32_t t = w * 16 + g * 4 + e;
      const float f = sc <= t ? expf((float)(bs[t] - bk)) : 0.0f;
      L[t][sc] = sc < t ? bet[t] * f * kk[j][e] : 0.0f;
      A[t][sc] = f * qq[j][e];
    }
  }
  __syncthreads();
  {  // the inverse of diagonal block w, column r16
    float x[16];
#pragma unroll
    for (int r = 0; r < 16; r++) {
      float v = r == (int)r16 ? 1.0f : 0.0f;
#pragma unroll
      for (int c = 0; c < r; c++) v = __builtin_fmaf(-L[w * 16 + r][w * 16 + c], x[c], v);
      x[r] = v;
      if (g == 0) T[w][r][r16] = v;
    }
  }
  __syncthreads();
  f32x4 lf[6], tf[4], af[10], be[4], bx[4];
#pragma unroll
  for (int i = 0; i < 4; i++) {
    tf[i] = *reinterpret_cast<const f32x4*>(&T[i][r16][g * 4]);
    be[i] = *reinterpret_cast<const f32x4*>(&bet[i * 16 + g * 4]);
    bx[i] = *reinterpret_cast<const f32x4*>(&eb[i * 16 + g * 4]);
#pragma unroll
    for (int j = 0; j <= i; j++) {
      af[i * (i + 1) / 2 + j] = *reinterpret_cast<const f32x4*>(&A[i * 16 + r16][j * 16 + g * 4]);
      if (j < i) lf[i * (i - 1) / 2 + j] = -*reinterpret_cast<const f32x4*>(&L[i * 16 + r16][j * 16 + g * 4]);
    }
  }
  const uint32_t nk = s.dk / 16, nt = nk + s.lv / 16;
  for (uint32_t ct = w; ct < nt; ct += 4) {                           // 16 columns of [keys | values]
    const bool key = ct < nk;                                         // (wave-uniform)
    const uint32_t c0 = (key ? ct : ct - nk) * 16;
    const float* src = (key ? K : b.v + ((size_t)t0 * s.heads + h) * s.lv) + c0;
    const size_t ld = key ? ldk : ldv;
    const uint32_t lo = (g * 4 * (uint32_t)ld + r16) * 4;
    f32x4 x[4], y[4];
#pragma unroll
    for (int i = 0; i < 4; i++)
#pragma unroll
      for (int e = 0; e < 4; e++) x[i][e] = at1(src, (i * 16 + e) * ld, lo);
#pragma unroll
    for (int i = 0; i < 4; i++) {
      x[i] *= key ? be[i] * bx[i] : be[i];
#pragma unroll
      for (int j = 0; j < i; j++) x[i] = Frag<float>::mma(lf[i * (i - 1) / 2 + j], x[j], x[i]);
      x[i] = Frag<float>::mma(tf[i], x[i], (f32x4)(0.0f));
    }
#pragma unroll
    for (int i = 0; i < 4; i++) {
      y[i] = (f32x4)(0.0f);
#pragma unroll
      for (int j = 0; j <= i; j++) y[i] = Frag<float>::mma(af[i * (i + 1) / 2 + j], x[j], y[i]);
    }
    const size_t at = (size_t)t0 * s.heads + h, ldo = key ? ldw : ldv;
    float* o0 = (key ? b.w + at * s.dk : b.u + at * s.lv) + c0;
    float* o1 = (key ? b.p + at * s.dk : b.num + at * s.lv) + c0;
    const uint32_t so = (g * 4 * (uint32_t)ldo + r16) * 4;
    if (key) {
      f32x4 z[4];
#pragma unroll
      for (int i = 0; i < 4; i++)
#pragma unroll
        for (int e = 0; e < 4; e++) z[i][e] = at1(Q + c0, (i * 16 + e) * ldk, lo);
#pragma unroll
      for (int i = 0; i < 4; i++) y[i] = bx[i] * z[i] - y[i];
    }
#pragma unroll
    for (int i = 0; i < 4; i++)
#pragma unroll
      for (int e = 0; e < 4; e++) {
        put1(o0, (i * 16 + e) * ldo, so, x[i][e]);
        put1(o1, (i * 16 + e) * ldo, so, y[i][e]);
      }
  }
}

// ------------------------------------------------------------------------------------------------
// blocks: the recurrence over the chunks; grid (heads, 16-column tiles): a head's tiles share an XCD where the heads are a multiple of 8.  Wave w of NW
// holds the state's rows NT * 16 * w .. as matrix-core accumulators; the waves' shares of W S and P S meet in LDS (one barrier per chunk).  PRE: the
// next chunk's operands are requested into registers while the current one is computed.
// ------------------------------------------------------------------------------------------------
template <int NT, int NW, bool PRE>
__global__ void __launch_bounds__(NW * 64, 1) delta_state_kernel(const DeltaShape s, const DeltaBufs b, uint32_t pos0, uint32_t nch) {
  extern __shared__ __attribute__((aligned(16))) f32x4 part[];         // [chunk parity][u, o][wave][token tile][lane]
  const uint32_t h = blockIdx.x, hk = h / (s.heads / s.kv_heads), c = blockIdx.y * 16 + (threadIdx.x & 15), lane = threadIdx.x & 63;
  const uint32_t w = (uint32_t)__builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6)), r16 = lane & 15, g = lane >> 4, dbase = w * NT * 16;
  const uint32_t ldk = s.kv_heads * s.dk, ldw = s.heads * s.dk, ldv = s.heads * s.lv;
  auto at = [&](uint32_t p, uint32_t k, uint32_t i, uint32_t j) -> f32x4& { return part[(((p * 2 + k) * NW + i) * 4 + j) * 64 + lane]; };
  float* Sg = b.S + (size_t)h * s.dk * s.lv + c;
  uint32_t dt[NT];                                                    // (tiles behind the last row repeat the first one, times 0)
  float live[NT];
  f32x4 S[NT];
#pragma unroll
  for (int i = 0; i < NT; i++) {
    const bool ok = dbase + i * 16 < s.dk;
    dt[i] = ok ? dbase + i * 16 : 0;
    live[i] = ok ? 1.0f : 0.0f;
#pragma unroll
    for (int e = 0; e < 4; e++) {
      const float v = Sg[(size_t)(dt[i] + g * 4 + e) * s.lv];
      S[i][e] = pos0 && ok ? v : 0.0f;
    }
  }
  const uint32_t lw = (r16 * ldw + g * 4) * 4, lk = (g * 4 * ldk + r16) * 4, lv = (g * 4 * ldv + r16) * 4;   // this lane's places
  const float* W0 = b.w + h * s.dk;
  const float* P0 = b.p + h * s.dk;
  const float* K0 = b.k + hk * s.dk;
  const float* U0 = b.u + h * s.lv + blockIdx.y * 16;
  float* O0 = b.num + h * s.lv + blockIdx.y * 16;
  struct Ops { f32x4 w[NT][4], p[NT][4], k[NT][4], u[4], wg[4], o; float cd; };
  auto fetch_s = [&](size_t t0, int i, Ops& x) {                      // what multiplies the state's tile i
#pragma unroll
    for (int j = 0; j < 4; j++) { x.w[i][j] = at4(W0, (t0 + j * 16) * ldw + dt[i], lw); x.p[i][j] = at4(P0, (t0 + j * 16) * ldw + dt[i], lw); }
  };
  auto fetch_k = [&](size_t t0, int i, Ops& x) {
#pragma unroll
    for (int j = 0; j < 4; j++)
#pragma unroll
      for (int e = 0; e < 4; e++) x.k[i][j][e] = at1(K0, (t0 + j * 16 + e) * ldk + dt[i], lk);
  };
  auto fetch_u = [&](uint32_t ch, Ops& x) {
    const size_t t0 = (size_t)ch * 64;
#pragma unroll
    for (int j = 0; j < 4; j++) {
#pragma unroll
      for (int e = 0; e < 4; e++) x.u[j][e] = at1(U0, (t0 + j * 16 + e) * ldv, lv);
      x.wg[j] = at4(b.wge + (size_t)h * b.Mcap, t0 + j * 16, g * 16);
    }
#pragma unroll
    for (int e = 0; e < 4; e++) x.o[e] = at1(O0, (t0 + (w & 3) * 16 + e) * ldv, lv);
    x.cd = b.cd[(size_t)h * (b.Mcap / 64) + ch];
  };
  auto fetch = [&](uint32_t ch, Ops& x) {
#pragma unroll
    for (int i = 0; i < NT; i++) { fetch_s((size_t)ch * 64, i, x); fetch_k((size_t)ch * 64, i, x); }
    fetch_u(ch, x);
  };
  auto chunk = [&](uint32_t ch, Ops& x) {
    f32x4 a[4], o[4];
#pragma unroll
    for (int j = 0; j < 4; j++) a[j] = o[j] = (f32x4)(0.0f);
    if (!PRE) fetch_u(ch, x);
#pragma unroll
    for (int i = 0; i < NT; i++) {
      if (!PRE) { fetch_s((size_t)ch * 64, i, x); asm volatile("" ::: "memory"); }   // (a tile's operands at a time: all of them do not fit the registers)
#pragma unroll
      for (int j = 0; j < 4; j++) a[j] = Frag<float>::mma(x.w[i][j], S[i], a[j]);
#pragma unroll
      for (int j = 0; j < 4; j++) o[j] = Frag<float>::mma(x.p[i][j], S[i], o[j]);
    }
#pragma unroll
    for (int j = 0; j < 4; j++) { at(ch & 1, 0, w, j) = a[j]; at(ch & 1, 1, w, j) = o[j]; }
    if (!PRE) fetch_k((size_t)ch * 64, 0, x);
    __syncthreads();
#pragma unroll
    for (int j = 0; j < 4; j++) {
      f32x4 t = at(ch & 1, 0, 0, j);
#pragma unroll
      for (int k = 1; k < NW; k++) t += at(ch & 1, 0, k, j);
      a[j] = (x.u[j] - t) * x.wg[j];
    }
#pragma unroll
    for (int i = 0; i < NT; i++) {
      if (!PRE && i + 1 < NT) { fetch_k((size_t)ch * 64, i + 1, x); asm volatile("" ::: "memory"); }
      S[i] *= x.cd;
#pragma unroll
      for (int j = 0; j < 4; j++) S[i] = Frag<float>::mma(x.k[i][j], a[j], S[i]);
      S[i] *= live[i];
    }
    if (w < 4) {                                                       // wave w finishes token tile w
      f32x4 t = at(ch & 1, 1, 0, w);
#pragma unroll
      for (int k = 1; k < NW; k++) t += at(ch & 1, 1, k, w);
      t += x.o;
#pragma unroll
      for (int e = 0; e < 4; e++) put1(O0, ((size_t)ch * 64 + w * 16 + e) * ldv, lv, t[e]);
    }
  };
  if constexpr (PRE) {
    Ops x0, x1;
    fetch(0, x0);
    for (uint32_t ch = 0; ch < nch; ch += 2) {
      fetch(ch + 1 < nch ? ch + 1 : ch, x1);
      chunk(ch, x0);
      if (ch + 1 >= nch) break;
      fetch(ch + 2 < nch ? ch + 2 : ch + 1, x0);
      chunk(ch + 1, x1);
    }
  } else {
    Ops x;
    for (uint32_t ch = 0; ch < nch; ch++) chunk(ch, x);
  }
#pragma unroll
  for (int i = 0; i < NT; i++)
#pragma unroll
    for (int e = 0; e < 4; e++)
      if (dbase + i * 16 < s.dk) Sg[(size_t)(dt[i] + g * 4 + e) * s.lv] = S[i][e];
}

template <int NT, int NW, bool PRE>
static hipError_t delta_state_go(const DeltaShape& s, const DeltaBufs& b, uint32_t pos0, uint32_t nch, hipStream_t st) {
  static bool opted[64] = {};
  constexpr size_t lds = (size_t)2 * 2 * NW * 4 * 64 * 16;
  if (hipError_t e = lds_opt_in(reinterpret_cast<const void*>(&delta_state_kernel<NT, NW, PRE>), (int)lds, opted); e != hipSuccess) return e;
  hipLaunchKernelGGL((delta_state_kernel<NT, NW, PRE>), dim3(s.heads, s.lv / 16), dim3(NW * 64), lds, st, s, b, pos0, nch);
  return hipGetLastError();
}

hipError_t delta_block_launch(const DeltaShape& s, const DeltaBufs& b, uint32_t pos0, uint32_t M, hipStream_t st) {
  const uint32_t nch = (M + 63) / 64;
  if (!delta_ok(s) || M == 0) return hipErrorInvalidValue;
  if (s.dim > kDeltaBlockDim) {   // a head's rows do not fit the state kernel's registers: the recurrence itself, token by token
    for (uint32_t t = 0; t < M; t++) {
      DeltaBufs r = b;
      r.cat += (size_t)t * s.ldcat;
      r.num += (size_t)t * s.heads * s.lv;
      if (hipError_t e = delta_step_launch(s, r, nullptr, pos0 + t, st); e != hipSuccess) return e;
    }
    return hipSuccess;
  }
  if (b.Mcap % 64 || nch * 64 > b.Mcap || !b.q || !b.k || !b.v || !b.u || !b.w || !b.p || !b.wge || !b.cd || 2 * s.kv_heads + s.heads > 65535) return hipErrorInvalidValue;
  const dim3 gp(nch * 2, 2 * s.kv_heads + s.heads), t(256);
  if (s.dk <= 64) hipLaunchKernelGGL(delta_prep_kernel<1>, gp, t, 0, st, s, b, pos0, M);
  else if (s.dk <= 128) hipLaunchKernelGGL(delta_prep_kernel<2>, gp, t, 0, st, s, b, pos0, M);
  else if (s.dk <= 256) hipLaunchKernelGGL(delta_prep_kernel<4>, gp, t, 0, st, s, b, pos0, M);
  else hipLaunchKernelGGL(delta_prep_kernel<8>, gp, t, 0, st, s, b, pos0, M);
  hipLaunchKernelGGL(delta_chunk_kernel, dim3(nch, s.heads), t, 0, st, s, b, M);
  if (hipError_t e = hipGetLastError(); e != hipSuccess) return e;
  if (s.dk <= 64) return delta_state_go<1, 4, true>(s, b, pos0, nch, st);
  if (s.dk <= 128) return delta_state_go<2, 4, true>(s, b, pos0, nch, st);
  if (s.dk <= 256) return delta_state_go<2, 8, false>(s, b, pos0, nch, st);
  return delta_state_go<4, 8, false>(s, b, pos0, nch, st);
}

// ------------------------------------------------------------------------------------------------
// grid: tokens, then one workgroup per row of the convolution's history that this block fills
// ------------------------------------------------------------------------------------------------
template <class T>
__global__ void __launch_bounds__(256) delta_out_kernel(const DeltaShape s, const DeltaBufs b, uint32_t pos0, uint32_t M, T* __restrict__ out, uint32_t ldo) {
  uint32_t t = blockIdx.x;
  if (t >= M) {
    t = M - 1 - (t - M);
    for (uint32_t c = threadIdx.x; c < s.cols; c += 256) b.hist[(size_t)((pos0 + t) % s.taps) * s.cols + c] = b.cat[(size_t)t * s.ldcat + c];
    return;
  }
  for (uint32_t h = threadIdx.x >> 6; h < s.heads; h += 4)
    head_read_out<T>(b.num + ((size_t)t * s.heads + h) * s.lv, b.norm, b.cat + (size_t)t * s.ldcat + s.off_g + (size_t)h * s.vdim, s.vdim, s.eps, 1.0f,
                     out + (size_t)t * ldo + (size_t)h * s.vdim);
}

hipError_t delta_out_launch(const DeltaShape& s, const DeltaBufs& b, uint32_t pos0, uint32_t M, void* out, uint32_t ldo, bool f32, hipStream_t st) {
  if (!delta_ok(s) || M == 0 || ldo < s.heads * s.vdim) return hipErrorInvalidValue;
  const dim3 grid(M + (M < s.taps ? M : s.taps));
  if (f32) hipLaunchKernelGGL(delta_out_kernel<float>, grid, dim3(256), 0, st, s, b, pos0, M, (float*)out, ldo);
  else hipLaunchKernelGGL(delta_out_kernel<__bf16>, grid, dim3(256), 0, st, s, b, pos0, M, (__bf16*)out, ldo);
  return hipGetLastError();
}

}  // namespace lgh
