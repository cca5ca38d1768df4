// mlstm.hip — the matrix-memory recurrence (mLSTM) of layered.h, all of it in 32-bit (exponents of the gates in 64-bit).
//
// With log forget gates f_t, log input gates i_t and the running maximum m_t = max(f_t + m_(t-1), i_t):
//   S_t = exp(f_t + m_(t-1) - m_t) S_(t-1) + exp(i_t - m_t) k_t v_t^T,   n_t the same with k_t alone,
//   o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6).
// n is kept as one more column of S (a value of constant 1), so a state is [head][dim][vdim + 1].
//
// Blocks of tokens use the recurrence's closed form.  With G_t = f_1 + .. + f_t (from the block's start), u_s = i_s - G_s and
// M_t = max(m_0, max_(s<=t) u_s):  m_t = G_t + M_t, the weight of token s in S_t is exp(u_s - M_t) and that of the state before the
// block exp(m_0 - M_t) — no exponent is ever positive.  64 tokens at a time:
//   numerators_t = exp(M_p - M_t) S_p^T q_t + sum_(s<=t) exp(u_s - M_t) (q_t . k_s) v_s        (p: the token before the chunk)
//   S_e = exp(M_p - M_e) S_p + sum_s exp(u_s - M_e) k_s v_s^T                                   (e: the chunk's last token)
// on the f32 matrix cores.  The chunk grid is relative to the block, so where a prompt is cut changes rounding only.
#include "layered.h"
#include "layered_device.h"

namespace lgh {

__device__ __forceinline__ float gate_in(float z, float cap) { return cap * tanhf(z / cap); }
__device__ __forceinline__ float log_sigmoid_f(float z) { return fminf(z, 0.0f) - log1pf(expf(-fabsf(z))); }

// ------------------------------------------------------------------------------------------------
// decode: one token.  A workgroup owns 32 columns of one head's state (8 lanes x 4 columns, 32 rows at a time).
// ------------------------------------------------------------------------------------------------
__global__ void __launch_bounds__(256) mlstm_step_kernel(const MlstmShape s, const MlstmBufs b, const int* __restrict__ pos_ptr) {
  __shared__ float o_s[32][33];
  const uint32_t h = blockIdx.y, tid = threadIdx.x, c4 = blockIdx.x * 32 + (tid & 7) * 4, r0 = tid >> 3;
  const uint32_t pos = (uint32_t)*pos_ptr;
  const float iv = gate_in(b.cat[s.off_i + h] + b.bi[h], s.cap);
  const float fv = log_sigmoid_f(gate_in(b.cat[s.off_f + h] + b.bf[h], s.cap));
  const double m0 = pos ? b.m[(pos & 1) * s.heads + h] : 0.0;
  const double m1 = fmax((double)fv + m0, (double)iv);
  const float fa = expf((float)((double)fv + m0 - m1)), fb = expf((float)((double)iv - m1));
  const float qs = 1.0f / __builtin_sqrtf((float)s.dim);
  const float* q = b.cat + s.off_q + (size_t)h * s.dim;
  const float* k = b.cat + s.off_k + (size_t)h * s.dim;
  const float* v = b.cat + s.off_v + (size_t)h * s.vdim;
  float vv[4], o[4];
#pragma unroll
  for (int e = 0; e < 4; e++) {
    const uint32_t c = c4 + e;
    vv[e] = fb * (c < s.vdim ? v[c] : c == s.vdim ? 1.0f : 0.0f);
    o[e] = 0.0f;
  }
  if (c4 < s.lds) {
    float* S = b.S + (size_t)h * s.dim * s.lds + c4;
#pragma unroll 4
    for (uint32_t d = r0; d < s.dim; d += 32) {
      f32x4* at = reinterpret_cast<f32x4*>(S + (size_t)d * s.lds);
      f32x4 st = (f32x4)(0.0f);
      if (pos) st = *at;
      const float kd = k[d], qd = q[d] * qs;
#pragma unroll
      for (int e = 0; e < 4; e++) {
        st[e] = __builtin_fmaf(kd, vv[e], fa * st[e]);
        o[e] = __builtin_fmaf(st[e], qd, o[e]);
      }
      *at = st;
    }
  }
#pragma unroll
  for (int e = 0; e < 4; e++) o_s[r0][(tid & 7) * 4 + e] = o[e];
  __syncthreads();
  if (tid < 32) {
    const uint32_t c = blockIdx.x * 32 + tid;
    float t = 0.0f;
    for (int r = 0; r < 32; r++) t += o_s[r][tid];
    if (c <= s.vdim) b.num[(size_t)h * s.ldo + c] = t;
    if (c == 0) {
      b.m[((pos + 1) & 1) * s.heads + h] = m1;
      b.num[(size_t)h * s.ldo + s.vdim + 1] = expf((float)(-m1));
    }
  }
}

hipError_t mlstm_step_launch(const MlstmShape& s, const MlstmBufs& b, const int* pos_ptr, hipStream_t st) {
  if (s.lds % 16 || s.lds < s.vdim + 1 || s.ldo < s.vdim + 2) return hipErrorInvalidValue;
  hipLaunchKernelGGL(mlstm_step_kernel, dim3((s.vdim + 1 + 31) / 32, s.heads), dim3(256), 0, st, s, b, pos_ptr);
  return hipGetLastError();
}

// ------------------------------------------------------------------------------------------------
// blocks of tokens: gates.  One wave per head, 64 tokens per step: a running sum (G) and a running maximum (M) across lanes.
// ------------------------------------------------------------------------------------------------
__global__ void __launch_bounds__(64) mlstm_gates_kernel(const MlstmShape s, const MlstmBufs b, uint32_t pos0, uint32_t M) {
  const uint32_t h = blockIdx.x, lane = threadIdx.x;
  const double m0 = pos0 ? b.m[(pos0 & 1) * s.heads + h] : 0.0;
  double G = 0.0, Mx = m0, mt = m0;
  const float bi = b.bi[h], bf = b.bf[h];
  for (uint32_t t0 = 0; t0 < M; t0 += 64) {
    const uint32_t t = t0 + lane;
    const bool ok = t < M;
    const float* row = b.cat + (size_t)(ok ? t : M - 1) * s.ldcat;
    const double iv = (double)gate_in(row[s.off_i + h] + bi, s.cap);
    double f = ok ? (double)log_sigmoid_f(gate_in(row[s.off_f + h] + bf, s.cap)) : 0.0;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) { const double p = __shfl_up(f, o, 64); if ((int)lane >= o) f += p; }
    const double Gt = G + f, u = iv - Gt;
    double mx = ok ? u : -1e300;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) { const double p = __shfl_up(mx, o, 64); if ((int)lane >= o) mx = fmax(mx, p); }
    mx = fmax(mx, Mx);
    if (ok) {
      b.u[(size_t)h * b.Mcap + t] = u;
      b.mx[(size_t)h * b.Mcap + t] = mx;
      b.num[((size_t)t * s.heads + h) * s.ldo + s.vdim + 1] = expf((float)(-(Gt + mx)));
    }
    G = __shfl(Gt, 63, 64);
    Mx = __shfl(mx, 63, 64);
    mt = G + Mx;
  }
  if (lane == 0) {
    b.m[((pos0 + M) & 1) * s.heads + h] = mt;   // (for an even M the half it was read from ...
    b.m[2 * s.heads + h] = m0;                  // ... so the state kernel finds the old value here)
  }
}

// four consecutive values p[0..3] of which the first n exist (n may be <= 0)
__device__ __forceinline__ f32x4 load4(const float* p, int n, bool vec) {
  if (vec && n >= 4) return *reinterpret_cast<const f32x4*>(p);
  f32x4 r = (f32x4)(0.0f);
#pragma unroll
  for (int e = 0; e < 4; e++)
    if (e < n) r[e] = p[e];
  return r;
}

// decayed scores of a chunk: A[t][s] = exp(u_s - M_t) (q_t . k_s) / sqrt(dim) for s <= t, else 0
__global__ void __launch_bounds__(256) mlstm_scores_kernel(const MlstmShape s, const MlstmBufs b, uint32_t M) {
  const uint32_t ch = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63, w = threadIdx.x >> 6, r16 = lane & 15, g = lane >> 4;
  const uint32_t t0 = ch * 64;
  const bool vec = (s.dim & 3) == 0 && (s.ldcat & 3) == 0 && (s.off_q & 3) == 0 && (s.off_k & 3) == 0;
  const float qs = 1.0f / __builtin_sqrtf((float)s.dim);
  const uint32_t tq = t0 + w * 16 + r16;
  const float* qrow = b.cat + (size_t)(tq < M ? tq : M - 1) * s.ldcat + s.off_q + (size_t)h * s.dim;
  const float* krow[4];
#pragma unroll
  for (int j = 0; j < 4; j++) {
    const uint32_t tk = t0 + j * 16 + r16;
    krow[j] = b.cat + (size_t)(tk < M ? tk : M - 1) * s.ldcat + s.off_k + (size_t)h * s.dim;
  }
  f32x4 acc[4];
#pragma unroll
  for (int j = 0; j < 4; j++) acc[j] = (f32x4)(0.0f);
  for (uint32_t d = 0; d < s.dim; d += 16) {
    const int n = (int)s.dim - (int)(d + g * 4);
    const f32x4 qf = load4(qrow + d + g * 4, n, vec);
#pragma unroll
    for (int j = 0; j < 4; j++)
      if (j <= (int)w) acc[j] = Frag<float>::mma(qf, load4(krow[j] + d + g * 4, n, vec), acc[j]);   // (wave-uniform: later keys are masked)
  }
  float* A = b.a + ((size_t)ch * s.heads + h) * 4096;
  const double* u = b.u + (size_t)h * b.Mcap;
  const double* mx = b.mx + (size_t)h * b.Mcap;
#pragma unroll
  for (int e = 0; e < 4; e++) {
    const uint32_t tl = w * 16 + g * 4 + e, t = t0 + tl;
    const double mt = t < M ? mx[t] : 0.0;
#pragma unroll
    for (int j = 0; j < 4; j++) {
      const uint32_t sl = j * 16 + r16;
      float v = 0.0f;
      if (t < M && sl <= tl) v = acc[j][e] * qs * expf((float)(u[t0 + sl] - mt));
      A[tl * 64 + sl] = v;
    }
  }
}

// the recurrence over the chunks.  A workgroup owns 16 columns of one head's state: wave w the rows of dim quarter w, as matrix-core
// accumulators (NT tiles of 16 rows).  A tile's register e of lane (column r16, group g) is row 4g + e — exactly what the j = e-th
// f32 product wants as its B operand, so the state is multiplied where it lies.
template <int NT>
__global__ void __launch_bounds__(256) mlstm_state_kernel(const MlstmShape s, const MlstmBufs b, uint32_t pos0, uint32_t M) {
  __shared__ f32x4 part[4][4][64];   // [wave][token tile][lane]
  const uint32_t h = blockIdx.y, c0 = blockIdx.x * 16, lane = threadIdx.x & 63;
  const uint32_t w = (uint32_t)__builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6));
  const uint32_t r16 = lane & 15, g = lane >> 4, c = c0 + r16;
  const bool vec = (s.dim & 3) == 0 && (s.ldcat & 3) == 0 && (s.off_q & 3) == 0;
  const float qs = 1.0f / __builtin_sqrtf((float)s.dim);
  const uint32_t dbase = w * NT * 16;
  const double* u = b.u + (size_t)h * b.Mcap;
  const double* mx = b.mx + (size_t)h * b.Mcap;
  float* Sg = b.S + (size_t)h * s.dim * s.lds;
  f32x4 S[NT];
#pragma unroll
  for (int i = 0; i < NT; i++)
#pragma unroll
    for (int e = 0; e < 4; e++) {
      const uint32_t d = dbase + i * 16 + g * 4 + e;
      S[i][e] = pos0 && d < s.dim && c <= s.vdim ? Sg[(size_t)d * s.lds + c] : 0.0f;
    }
  double mp = b.m[2 * s.heads + h];
  const uint32_t nch = (M + 63) / 64;
  for (uint32_t ch = 0; ch < nch; ch++) {
    const uint32_t t0 = ch * 64, te = (t0 + 63 < M ? t0 + 63 : M - 1);
    const double me = mx[te];
    // ---- numerators: the wave's share of S^T q (its dim quarter) and of A v (its 16 source tokens)
    f32x4 o[4];
#pragma unroll
    for (int j = 0; j < 4; j++) o[j] = (f32x4)(0.0f);
#pragma unroll
    for (int i = 0; i < NT; i++) {
      const uint32_t d = dbase + i * 16 + g * 4;
#pragma unroll
      for (int j = 0; j < 4; j++) {
        const uint32_t t = t0 + j * 16 + r16;
        const f32x4 qf = load4(b.cat + (size_t)(t < M ? t : M - 1) * s.ldcat + s.off_q + (size_t)h * s.dim + d, (int)s.dim - (int)d, vec);
        o[j] = Frag<float>::mma(qf, S[i], o[j]);
      }
    }
#pragma unroll
    for (int j = 0; j < 4; j++)
#pragma unroll
      for (int e = 0; e < 4; e++) {
        const uint32_t t = t0 + j * 16 + g * 4 + e;
        o[j][e] *= qs * expf((float)(mp - (t < M ? mx[t] : me)));
      }
    f32x4 vf;                                                   // v of the wave's 16 tokens: lane column c, tokens 4g .. 4g + 3
#pragma unroll
    for (int e = 0; e < 4; e++) {
      const uint32_t t = t0 + w * 16 + g * 4 + e;
      vf[e] = t < M ? (c < s.vdim ? b.cat[(size_t)t * s.ldcat + s.off_v + (size_t)h * s.vdim + c] : c == s.vdim ? 1.0f : 0.0f) : 0.0f;
    }
    const float* A = b.a + ((size_t)ch * s.heads + h) * 4096;
#pragma unroll
    for (int j = 0; j < 4; j++)
      if (j >= (int)w) o[j] = Frag<float>::mma(*reinterpret_cast<const f32x4*>(A + (j * 16 + r16) * 64 + w * 16 + g * 4), vf, o[j]);
#pragma unroll
    for (int j = 0; j < 4; j++) part[w][j][lane] = o[j];
    // ---- the state at the chunk's end
    const float decay = expf((float)(mp - me));
#pragma unroll
    for (int i = 0; i < NT; i++) S[i] *= decay;
#pragma unroll
    for (int sj = 0; sj < 4; sj++) {
      if (t0 + sj * 16 >= M) break;
      f32x4 wv;
      uint32_t tt[4];
#pragma unroll
      for (int e = 0; e < 4; e++) {
        const uint32_t t = t0 + sj * 16 + g * 4 + e;
        tt[e] = t < M ? t : M - 1;
        const float v = c < s.vdim ? b.cat[(size_t)tt[e] * s.ldcat + s.off_v + (size_t)h * s.vdim + c] : c == s.vdim ? 1.0f : 0.0f;
        wv[e] = t < M ? v * expf((float)(u[t] - me)) : 0.0f;
      }
#pragma unroll
      for (int i = 0; i < NT; i++) {
        const uint32_t d = dbase + i * 16 + r16;
        f32x4 kf = (f32x4)(0.0f);
        if (d < s.dim) {
#pragma unroll
          for (int e = 0; e < 4; e++) kf[e] = b.cat[(size_t)tt[e] * s.ldcat + s.off_k + (size_t)h * s.dim + d];
        }
        S[i] = Frag<float>::mma(kf, wv, S[i]);
      }
    }
    mp = me;
    __syncthreads();
    {  // add the four waves' shares; wave w finishes token tile w
      const f32x4 t4 = (part[0][w][lane] + part[1][w][lane]) + (part[2][w][lane] + part[3][w][lane]);
#pragma unroll
      for (int e = 0; e < 4; e++) {
        const uint32_t t = t0 + w * 16 + g * 4 + e;
        if (t < M && c <= s.vdim) b.num[((size_t)t * s.heads + h) * s.ldo + c] = t4[e];
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < NT; i++)
#pragma unroll
    for (int e = 0; e < 4; e++) {
      const uint32_t d = dbase + i * 16 + g * 4 + e;
      if (d < s.dim && c <= s.vdim) Sg[(size_t)d * s.lds + c] = S[i][e];
    }
}

hipError_t mlstm_block_launch(const MlstmShape& s, const MlstmBufs& b, uint32_t pos0, uint32_t M, hipStream_t st) {
  if (M == 0 || M > b.Mcap || s.dim > kMlstmMaxDim || s.lds < s.vdim + 1 || s.ldo < s.vdim + 2) return hipErrorInvalidValue;
  const dim3 gs((s.vdim + 1 + 15) / 16, s.heads), t(256);
  hipLaunchKernelGGL(mlstm_gates_kernel, dim3(s.heads), dim3(64), 0, st, s, b, pos0, M);
  hipLaunchKernelGGL(mlstm_scores_kernel, dim3((M + 63) / 64, s.heads), t, 0, st, s, b, M);
  const uint32_t nt = (s.dim + 63) / 64;
  if (nt <= 1) hipLaunchKernelGGL(mlstm_state_kernel<1>, gs, t, 0, st, s, b, pos0, M);
  else if (nt <= 2) hipLaunchKernelGGL(mlstm_state_kernel<2>, gs, t, 0, st, s, b, pos0, M);
  else if (nt <= 4) hipLaunchKernelGGL(mlstm_state_kernel<4>, gs, t, 0, st, s, b, pos0, M);
  else if (nt <= 8) hipLaunchKernelGGL(mlstm_state_kernel<8>, gs, t, 0, st, s, b, pos0, M);
  else hipLaunchKernelGGL(mlstm_state_kernel<16>, gs, t, 0, st, s, b, pos0, M);
  return hipGetLastError();
}

// ------------------------------------------------------------------------------------------------
// read-out of a block: numerators / denominators, per-head RMS norm, norm weight, sigmoid gate -> activations.  A wave per head.
// ------------------------------------------------------------------------------------------------
template <class T>
__global__ void __launch_bounds__(256) mlstm_out_kernel(const MlstmShape s, const MlstmBufs b, T* __restrict__ out, uint32_t ldo) {
  const uint32_t t = blockIdx.x, lane = threadIdx.x & 63;
  for (uint32_t h = threadIdx.x >> 6; h < s.heads; h += 4) {
    const float* num = b.num + ((size_t)t * s.heads + h) * s.ldo;
    const float inv = 1.0f / (fmaxf(fabsf(num[s.vdim]), num[s.vdim + 1]) + 1e-6f);
    float ss = 0.0f;
    for (uint32_t j = lane; j < s.vdim; j += 64) { const float o = num[j] * inv; ss = __builtin_fmaf(o, o, ss); }
    const float r = 1.0f / __builtin_sqrtf(wave_sum(ss) / (float)s.vdim + s.eps);
    const float* gate = b.cat + (size_t)t * s.ldcat + s.off_g + (size_t)h * s.vdim;
    for (uint32_t j = lane; j < s.vdim; j += 64)
      out[(size_t)t * ldo + h * s.vdim + j] = to_act<T>(num[j] * inv * r * b.norm[h * s.vdim + j] * sigmoid_f(gate[j]));
  }
}

hipError_t mlstm_out_launch(const MlstmShape& s, const MlstmBufs& b, uint32_t M, void* out, uint32_t ldo, bool f32, hipStream_t st) {
  if (f32) hipLaunchKernelGGL(mlstm_out_kernel<float>, dim3(M), dim3(256), 0, st, s, b, (float*)out, ldo);
  else hipLaunchKernelGGL(mlstm_out_kernel<__bf16>, dim3(M), dim3(256), 0, st, s, b, (__bf16*)out, ldo);
  return hipGetLastError();
}

}  // namespace lgh
