// mlstm.hip — the matrix-memory recurrence (mLSTM) of layered.h, all of it in 32-bit (exponents of the gates in 64-bit).
//
// With log forget gates f_t, log input gates i_t and the running maximum m_t = max(f_t + m_(t-1), i_t):
//   S_t = exp(f_t + m_(t-1) - m_t) S_(t-1) + exp(i_t - m_t) k_t v_t^T,   n_t the same with k_t alone,
//   o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6).
// n is kept as one more column of S (a value of constant 1), so a state is [head][dim][vdim + 1]; the block kernels take it apart (the
// state kernel's workgroups are one per CU at common sizes, a 16-column tile of n alone would be a second round).
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

// ------------------------------------------------------------------------------------------------
// decode: one token.  A workgroup owns 16 columns of one head's state (4 lanes x 4 columns, 64 rows at a time).
// ------------------------------------------------------------------------------------------------
__global__ void __launch_bounds__(256) mlstm_step_kernel(const MlstmShape s, const MlstmBufs b, const int* __restrict__ pos_ptr, uint32_t pos0) {
  __shared__ float o_s[4][16];
  const uint32_t h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, c4 = blockIdx.x * 16 + (tid & 3) * 4, r0 = tid >> 2;
  const uint32_t pos = pos_ptr ? (uint32_t)*pos_ptr : pos0;
  const float* q = b.cat + s.off_q + (size_t)h * s.dim;
  const float* k = b.cat + s.off_k + (size_t)h * s.dim;
  const float* v = b.cat + s.off_v + (size_t)h * s.vdim;
  float* S = b.S + (size_t)h * s.dim * s.lds + c4;
  f32x4 st[4];
  float kd[4], qd[4];
  auto fetch = [&](uint32_t d0) {   // 4 x 64 rows (rows past the end re-read the last one and are dropped)
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const uint32_t d = d0 + i * 64 + r0, dc = d < s.dim ? d : s.dim - 1;
      st[i] = *reinterpret_cast<const f32x4*>(S + (size_t)dc * s.lds);
      kd[i] = k[dc];
      qd[i] = q[dc];
    }
  };
  fetch(0);
  const float iv = gate_in(b.cat[s.off_i + h] + b.bi[h], s.cap);
  const float fv = log_sigmoid_f(gate_in(b.cat[s.off_f + h] + b.bf[h], s.cap));
  const double m0 = pos ? b.m[(pos & 1) * s.heads + h] : 0.0;
  const double m1 = fmax((double)fv + m0, (double)iv);
  const float fa = expf((float)((double)fv + m0 - m1)), fb = expf((float)((double)iv - m1));
  const float qs = 1.0f / __builtin_sqrtf((float)s.dim);
  float vv[4], o[4];
#pragma unroll
  for (int e = 0; e < 4; e++) {
    const uint32_t c = c4 + e;
    vv[e] = fb * (c < s.vdim ? v[c] : c == s.vdim ? 1.0f : 0.0f);
    o[e] = 0.0f;
  }
  for (uint32_t d0 = 0; d0 < s.dim; d0 += 256) {
    if (d0) fetch(d0);
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const uint32_t d = d0 + i * 64 + r0;
      if (d >= s.dim) continue;
      f32x4 x;
#pragma unroll
      for (int e = 0; e < 4; e++) {
        x[e] = __builtin_fmaf(kd[i], vv[e], pos ? fa * st[i][e] : 0.0f);   // at position 0 whatever is stored belongs to another sequence
        o[e] = __builtin_fmaf(x[e], qd[i], o[e]);
      }
      *reinterpret_cast<f32x4*>(S + (size_t)d * s.lds) = x;
    }
  }
#pragma unroll
  for (int e = 0; e < 4; e++) {   // the 16 row slots of a wave: lanes with equal lane & 3
    o[e] *= qs;
    o[e] += __shfl_xor(o[e], 4, 64); o[e] += __shfl_xor(o[e], 8, 64); o[e] += __shfl_xor(o[e], 16, 64); o[e] += __shfl_xor(o[e], 32, 64);
    if (lane < 4) o_s[tid >> 6][lane * 4 + e] = o[e];
  }
  __syncthreads();
  if (tid < 16) {
    const uint32_t c = blockIdx.x * 16 + tid;
    if (c <= s.vdim) b.num[(size_t)h * s.ldo + c] = (o_s[0][tid] + o_s[1][tid]) + (o_s[2][tid] + o_s[3][tid]);
    if (c == 0) {
      b.m[((pos + 1) & 1) * s.heads + h] = m1;
      b.num[(size_t)h * s.ldo + s.vdim + 1] = expf((float)(-m1));
    }
  }
}

hipError_t mlstm_step_launch(const MlstmShape& s, const MlstmBufs& b, const int* pos_ptr, hipStream_t st, uint32_t pos0) {
  if (s.lds % 16 || s.lds < s.vdim + 1 || s.ldo < s.vdim + 2) return hipErrorInvalidValue;
  hipLaunchKernelGGL(mlstm_step_kernel, dim3((s.vdim + 1 + 15) / 16, s.heads), dim3(256), 0, st, s, b, pos_ptr, pos0);
  return hipGetLastError();
}

// ------------------------------------------------------------------------------------------------
// blocks of tokens: gates.  One workgroup per head; a wave takes one chunk of 64 tokens at a time (16 chunks a round) and scans it from
// the chunk's own start — a running sum (G) and a running maximum (of u) across lanes; the chunks' offsets then follow in order.
// Besides u and M it leaves, as f32 factors for the state kernel: dec_t = exp(M_p - M_t) / sqrt(dim), wgt_t = exp(u_t - M_e) and each
// chunk's exp(M_p - M_e) (p: the token before the chunk, e: its last token).
// ------------------------------------------------------------------------------------------------
__global__ void __launch_bounds__(1024) mlstm_gates_kernel(const MlstmShape s, const MlstmBufs b, uint32_t pos0, uint32_t M) {
  __shared__ double tot[16], top[16], G0[17], M0[17];
  const uint32_t h = blockIdx.x, lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const double m0 = pos0 ? b.m[(pos0 & 1) * s.heads + h] : 0.0;
  const float bi = b.bi[h], bf = b.bf[h];
  const float qs = 1.0f / __builtin_sqrtf((float)s.dim);
  double G = 0.0, Mx = m0;
  for (uint32_t base = 0; base < M; base += 1024) {
    const uint32_t t = base + w * 64 + lane;
    const bool ok = t < M;
    const float* row = b.cat + (size_t)(ok ? t : M - 1) * s.ldcat;
    const double iv = (double)gate_in(row[s.off_i + h] + bi, s.cap);
    double f = ok ? (double)log_sigmoid_f(gate_in(row[s.off_f + h] + bf, s.cap)) : 0.0;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) { const double p = __shfl_up(f, o, 64); if ((int)lane >= o) f += p; }
    const double ul = iv - f;                     // u up to the chunk's offset
    double mx = ok ? ul : -1e300;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) { const double p = __shfl_up(mx, o, 64); if ((int)lane >= o) mx = fmax(mx, p); }
    if (lane == 63) { tot[w] = f; top[w] = mx; }
    __syncthreads();
    if (threadIdx.x == 0) {
      double g = G, m = Mx;
      for (int i = 0; i < 16; i++) {
        G0[i] = g; M0[i] = m;
        m = fmax(m, top[i] - g);
        g += tot[i];
      }
      G0[16] = g; M0[16] = m;
    }
    __syncthreads();
    const double g0 = G0[w], mp = M0[w], me = M0[w + 1];
    const double u = ul - g0, mt = fmax(mp, mx - g0);
    if (!ok && t < ((M + 63) & ~63u)) b.wgt[(size_t)h * b.Mcap + t] = 0.0f;   // the rest of the last chunk
    if (ok) {
      const size_t at = (size_t)h * b.Mcap + t;
      b.u[at] = u;
      b.mx[at] = mt;
      b.dec[at] = qs * expf((float)(mp - mt));
      b.wgt[at] = expf((float)(u - me));
      if (lane == 0) b.cdec[(size_t)h * (b.Mcap / 64) + t / 64] = expf((float)(mp - me));
      b.num[((size_t)t * s.heads + h) * s.ldo + s.vdim + 1] = expf((float)(-(g0 + f + mt)));
    }
    G = G0[16];
    Mx = M0[16];
  }
  if (threadIdx.x == 0) b.m[((pos0 + M) & 1) * s.heads + h] = G + Mx;
}

// Loads of the block kernels are unconditional and masks are factors (a select with a loaded operand becomes a branch around the load,
// which then waits for it): a head's last 16-wide tile may read on into the next head's or segment's values — the row buffer has room for
// that behind its last row — and one side of every product is multiplied by 0 there.
template <bool VEC>   // VEC: rows and heads start at multiples of 16 bytes
__device__ __forceinline__ f32x4 row4(const float* base, uint32_t off) {
  const char* p = reinterpret_cast<const char*>(base) + off * 4u;
  if constexpr (VEC) return *reinterpret_cast<const f32x4*>(p);
  f32x4 r;
#pragma unroll
  for (int e = 0; e < 4; e++) r[e] = *reinterpret_cast<const float*>(p + 4 * e);
  return r;
}
__device__ __forceinline__ float row1(const float* base, uint32_t off) { return *reinterpret_cast<const float*>(reinterpret_cast<const char*>(base) + off * 4u); }
// the four values at dims d .. d + 3 of a query, zero from dim on
__device__ __forceinline__ f32x4 keep_dims(f32x4 v, uint32_t d, uint32_t dim) {
#pragma unroll
  for (int e = 0; e < 4; e++) v[e] *= d + e < dim ? 1.0f : 0.0f;
  return v;
}

// decayed scores of a chunk: A[t][s] = exp(u_s - M_t) (q_t . k_s) / sqrt(dim) for s <= t, else 0
template <bool VEC>
__global__ void __launch_bounds__(256) mlstm_scores_kernel(const MlstmShape s, const MlstmBufs b, uint32_t M) {
  const uint32_t ch = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63, w = threadIdx.x >> 6, r16 = lane & 15, g = lane >> 4;
  const uint32_t t0 = ch * 64;
  const float qs = 1.0f / __builtin_sqrtf((float)s.dim);
  const uint32_t tq = t0 + w * 16 + r16;
  const uint32_t qo = (tq < M ? tq : M - 1) * s.ldcat + s.off_q + h * s.dim + g * 4;
  uint32_t ko[4];
#pragma unroll
  for (int j = 0; j < 4; j++) {
    const uint32_t tk = t0 + j * 16 + r16;
    ko[j] = (tk < M ? tk : M - 1) * s.ldcat + s.off_k + h * s.dim + g * 4;
  }
  f32x4 acc[4];
#pragma unroll
  for (int j = 0; j < 4; j++) acc[j] = (f32x4)(0.0f);
  for (uint32_t d = 0; d < s.dim; d += 16) {
    const f32x4 qf = keep_dims(row4<VEC>(b.cat, qo + d), d + g * 4, s.dim);
#pragma unroll
    for (int j = 0; j < 4; j++) acc[j] = Frag<float>::mma(qf, row4<VEC>(b.cat, ko[j] + d), acc[j]);
  }
  {  // the chunk's contribution to n: sum_s exp(u_s - M_e) k_s
    const uint32_t rows = M - t0 < 64 ? M - t0 : 64;
    const float* wg = b.wgt + (size_t)h * b.Mcap + t0;
    for (uint32_t d = threadIdx.x; d < s.dim; d += 256) {
      float n = 0.0f;
#pragma unroll 8
      for (uint32_t r = 0; r < rows; r++) n = __builtin_fmaf(wg[r], row1(b.cat, (t0 + r) * s.ldcat + s.off_k + h * s.dim + d), n);
      b.nk[((size_t)ch * s.heads + h) * s.dim + d] = n;
    }
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

// n before every chunk (in place of the chunks' contributions) and after the last
__global__ void __launch_bounds__(256) mlstm_n_kernel(const MlstmShape s, const MlstmBufs b, uint32_t pos0, uint32_t M) {
  const uint32_t h = blockIdx.y, d = blockIdx.x * 256 + threadIdx.x, nch = (M + 63) / 64;
  if (d >= s.dim) return;
  float* Sn = b.S + ((size_t)h * s.dim + d) * s.lds + s.vdim;
  const float* cdec = b.cdec + (size_t)h * (b.Mcap / 64);
  float n = pos0 ? *Sn : 0.0f;
  for (uint32_t c0 = 0; c0 < nch; c0 += 8) {
    float k[8], f[8];
#pragma unroll
    for (uint32_t i = 0; i < 8; i++) {
      const uint32_t ch = c0 + i < nch ? c0 + i : nch - 1;
      k[i] = b.nk[((size_t)ch * s.heads + h) * s.dim + d];
      f[i] = cdec[ch];
    }
#pragma unroll
    for (uint32_t i = 0; i < 8; i++)
      if (c0 + i < nch) {
        b.nk[((size_t)(c0 + i) * s.heads + h) * s.dim + d] = n;
        n = __builtin_fmaf(f[i], n, k[i]);
      }
  }
  *Sn = n;
}

// the recurrence over the chunks.  A workgroup owns 16 columns of one head's state: wave w of NW the rows NT * 16 * w .., as matrix-core
// accumulators (NT tiles of 16 rows).  A tile's register e of lane (column r16, group g) is row 4g + e — exactly what the j = e-th
// f32 product wants as its B operand, so the state is multiplied where it lies.  The workgroups are few (one per CU and less), so the
// next chunk's operands are requested into registers while the current one is computed (PRE; large dims have no registers for it).
// ROWS: queries and keys carry their decays already, and the state's rows decay each at its own rate (rowdec).
template <int NT, int NW, bool PRE, bool VEC, bool ROWS>
__global__ void __launch_bounds__(NW * 64, 1) mlstm_state_kernel(const MlstmShape s, const MlstmBufs b, uint32_t pos0, uint32_t M) {
  __shared__ f32x4 part[2][NW][4][64];   // [chunk parity][wave][token tile][lane]
  const uint32_t h = blockIdx.y, c0 = blockIdx.x * 16, lane = threadIdx.x & 63;
  const uint32_t w = (uint32_t)__builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6));
  const uint32_t r16 = lane & 15, g = lane >> 4, c = c0 + r16;
  const uint32_t dbase = w * NT * 16;
  const float* dec = b.dec + (size_t)h * b.Mcap;
  const float* wgt = b.wgt + (size_t)h * b.Mcap;
  const float* cdec = ROWS ? nullptr : b.cdec + (size_t)h * (b.Mcap / 64);
  float* Sg = b.S + (size_t)h * s.dim * s.lds;
  const uint32_t qo = s.off_q + h * s.dim + dbase + g * 4, ko = s.off_k + h * s.dim + dbase + r16, vo = s.off_v + h * s.vdim + (c < s.vdim ? c : 0);
  const bool ragged = s.dim != NT * NW * 16;   // rows past dim: never stored, kept 0
  f32x4 S[NT];
#pragma unroll
  for (int i = 0; i < NT; i++)
#pragma unroll
    for (int e = 0; e < 4; e++) {
      const uint32_t d = dbase + i * 16 + g * 4 + e;
      const bool ok = d < s.dim && c < s.vdim;
      const float v = Sg[ok ? (size_t)d * s.lds + c : 0];
      S[i][e] = pos0 && ok ? v : 0.0f;
    }
  struct Ops { f32x4 q[NT][4]; f32x4 k[NT][4]; f32x4 v[4], wg[4], dc[4], a[4], rd[ROWS ? NT : 1]; float cd; };
  // a chunk's operands: q tiles (lane: token r16 of tile j, 4 dims), k (lane: dim r16, tokens 4g ..), v, factors, the wave's score columns.
  // Tokens past the end re-read the last one: their weight is 0 and their numerators are not stored.
  auto fetch = [&](uint32_t ch, Ops& x) {
    const uint32_t t0 = ch * 64;
#pragma unroll
    for (int j = 0; j < 4; j++) {
      const uint32_t t = t0 + j * 16 + r16, ro = (t < M ? t : M - 1) * s.ldqk + qo;
#pragma unroll
      for (int i = 0; i < NT; i++) x.q[i][j] = row4<VEC>(b.qk, ro + i * 16);
#pragma unroll
      for (int e = 0; e < 4; e++) {
        const uint32_t ts = t0 + j * 16 + g * 4 + e, tsc = ts < M ? ts : M - 1;
        x.v[j][e] = row1(b.cat, tsc * s.ldcat + vo);   // (columns past vdim: computed, never stored)
        if constexpr (!ROWS) {
          x.wg[j][e] = row1(wgt, ts);   // (0 behind the block's last token)
          x.dc[j][e] = row1(dec, tsc);
        }
#pragma unroll
        for (int i = 0; i < NT; i++) x.k[i][j][e] = row1(b.qk, (ROWS ? ts : tsc) * s.ldqk + ko + i * 16);   // (ROWS: zeros behind the last token)
      }
      x.a[j] = *reinterpret_cast<const f32x4*>(b.a + ((size_t)ch * s.heads + h) * 4096 + (j * 16 + r16) * 64 + (w & 3) * 16 + g * 4);
    }
    if constexpr (ROWS) {
#pragma unroll
      for (int i = 0; i < NT; i++) x.rd[i] = row4<VEC>(b.rowdec, (ch * s.heads + h) * s.dim + dbase + g * 4 + i * 16);
    } else {
      x.cd = cdec[ch];
    }
  };
  auto chunk = [&](uint32_t ch, const Ops& x) {
    const uint32_t t0 = ch * 64;
    f32x4 o[4];
#pragma unroll
    for (int j = 0; j < 4; j++) o[j] = (f32x4)(0.0f);
    // numerators: the wave's share of S^T q (its rows) and of A v (16 source tokens; the first four waves)
#pragma unroll
    for (int i = 0; i < NT; i++)
#pragma unroll
      for (int j = 0; j < 4; j++) o[j] = Frag<float>::mma(x.q[i][j], S[i], o[j]);
    f32x4 vw;
#pragma unroll
    for (int e = 0; e < 4; e++) {
      const float v = w == 0 ? x.v[0][e] : w == 1 ? x.v[1][e] : w == 2 ? x.v[2][e] : x.v[3][e];
      vw[e] = v;
    }
#pragma unroll
    for (int j = 0; j < 4; j++) {
      if constexpr (!ROWS) o[j] *= x.dc[j];
      if (w < 4) o[j] = Frag<float>::mma(x.a[j], vw, o[j]);   // (scores of later keys are stored as zeros)
      part[ch & 1][w][j][lane] = o[j];
    }
    // the state at the chunk's end
#pragma unroll
    for (int i = 0; i < NT; i++) {
      if constexpr (ROWS) S[i] *= x.rd[i];
      else S[i] *= x.cd;
    }
#pragma unroll
    for (int j = 0; j < 4; j++) {
      const f32x4 wv = ROWS ? x.v[j] : x.v[j] * x.wg[j];
#pragma unroll
      for (int i = 0; i < NT; i++) S[i] = Frag<float>::mma(x.k[i][j], wv, S[i]);
    }
    if (ragged) {
#pragma unroll
      for (int i = 0; i < NT; i++)
#pragma unroll
        for (int e = 0; e < 4; e++) S[i][e] *= dbase + i * 16 + g * 4 + e < s.dim ? 1.0f : 0.0f;
    }
    __syncthreads();
    if (w >= 4) return;
    f32x4 t4 = (part[ch & 1][0][w][lane] + part[ch & 1][1][w][lane]) + (part[ch & 1][2][w][lane] + part[ch & 1][3][w][lane]);
#pragma unroll
    for (int k = 4; k < NW; k++) t4 += part[ch & 1][k][w][lane];
#pragma unroll
    for (int e = 0; e < 4; e++) {   // wave w finishes token tile w
      const uint32_t t = t0 + w * 16 + g * 4 + e;
      if (t < M && c < s.vdim) b.num[((size_t)t * s.heads + h) * s.ldo + c] = t4[e];
    }
  };
  const uint32_t nch = (M + 63) / 64;
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
    for (uint32_t ch = 0; ch < nch; ch++) {
      fetch(ch, x);
      chunk(ch, x);
    }
  }
#pragma unroll
  for (int i = 0; i < NT; i++)
#pragma unroll
    for (int e = 0; e < 4; e++) {
      const uint32_t d = dbase + i * 16 + g * 4 + e;
      if (d < s.dim && c < s.vdim) Sg[(size_t)d * s.lds + c] = S[i][e];
    }
}

hipError_t mlstm_block_launch(const MlstmShape& s, const MlstmBufs& b, uint32_t pos0, uint32_t M, hipStream_t st) {
  if (M == 0 || M > b.Mcap || b.Mcap % 64 || s.lds < s.vdim + 1 || s.ldo < s.vdim + 2) return hipErrorInvalidValue;
  if (s.dim > kMlstmBlockDim) {   // a head's rows do not fit the block kernel's registers: the recurrence itself, token by token
    for (uint32_t t = 0; t < M; t++) {
      MlstmBufs r = b;
      r.cat += (size_t)t * s.ldcat;
      r.num += (size_t)t * s.heads * s.ldo;
      if (hipError_t e = mlstm_step_launch(s, r, nullptr, st, pos0 + t); e != hipSuccess) return e;
    }
    return hipSuccess;
  }
  const dim3 t(256);
  hipLaunchKernelGGL(mlstm_gates_kernel, dim3(s.heads), dim3(1024), 0, st, s, b, pos0, M);
  const bool vec = (s.dim & 3) == 0 && (s.ldcat & 3) == 0 && (s.off_q & 3) == 0 && (s.off_k & 3) == 0;
  const dim3 gq((M + 63) / 64, s.heads);
  if (vec) hipLaunchKernelGGL(mlstm_scores_kernel<true>, gq, t, 0, st, s, b, M);
  else hipLaunchKernelGGL(mlstm_scores_kernel<false>, gq, t, 0, st, s, b, M);
  hipLaunchKernelGGL(mlstm_n_kernel, dim3((s.dim + 255) / 256, s.heads), t, 0, st, s, b, pos0, M);
  return mlstm_state_launch(s, b, pos0, M, st);
}

template <bool VEC, bool ROWS>
static hipError_t mlstm_state_go(const MlstmShape& s, const MlstmBufs& b, uint32_t pos0, uint32_t M, hipStream_t st) {
  const uint32_t nt = (s.dim + 63) / 64;
  const dim3 gs((s.vdim + 15) / 16, s.heads);
#define LGH_STATE(N, W, P) hipLaunchKernelGGL((mlstm_state_kernel<N, W, P, VEC, ROWS>), gs, dim3(W * 64), 0, st, s, b, pos0, M)
  if (nt <= 1) LGH_STATE(1, 4, true);
  else if (nt <= 2) LGH_STATE(2, 4, true);
  else if (nt <= 4) LGH_STATE(4, 4, true);
  else LGH_STATE(4, 8, false);
#undef LGH_STATE
  return hipGetLastError();
}

hipError_t mlstm_state_launch(const MlstmShape& s, const MlstmBufs& b, uint32_t pos0, uint32_t M, hipStream_t st) {
  if (M == 0 || M > b.Mcap || b.Mcap % 64 || s.dim > kMlstmBlockDim || !b.qk || s.lds < s.vdim) return hipErrorInvalidValue;
  const bool vec = (s.dim & 3) == 0 && (s.ldqk & 3) == 0 && (s.off_q & 3) == 0 && (s.off_k & 3) == 0;
  if (b.rowdec) return vec ? mlstm_state_go<true, true>(s, b, pos0, M, st) : mlstm_state_go<false, true>(s, b, pos0, M, st);
  return vec ? mlstm_state_go<true, false>(s, b, pos0, M, st) : mlstm_state_go<false, false>(s, b, pos0, M, st);
}

// ------------------------------------------------------------------------------------------------
// read-out of a block: numerators / denominators, per-head RMS norm, norm weight, sigmoid gate -> activations.  A wave per head.
// ------------------------------------------------------------------------------------------------
template <class T>
__global__ void __launch_bounds__(256) mlstm_out_kernel(const MlstmShape s, const MlstmBufs b, T* __restrict__ out, uint32_t ldo) {
  const uint32_t t = blockIdx.x, lane = threadIdx.x & 63;
  for (uint32_t h = threadIdx.x >> 6; h < s.heads; h += 4) {
    const float* num = b.num + ((size_t)t * s.heads + h) * s.ldo;
    float den;
    if (s.dim > kMlstmBlockDim) {
      den = num[s.vdim];
    } else {   // n . q = exp(M_p - M_t) n_p . q + the row sum of the decayed scores
      const size_t chh = (size_t)(t / 64) * s.heads + h;
      const float* q = b.cat + (size_t)t * s.ldcat + s.off_q + (size_t)h * s.dim;
      const float* n = b.nk + chh * s.dim;
      float dot = 0.0f;
      for (uint32_t d = lane; d < s.dim; d += 64) dot = __builtin_fmaf(q[d], n[d], dot);
      den = wave_sum(__builtin_fmaf(dot, b.dec[(size_t)h * b.Mcap + t], b.a[chh * 4096 + (t & 63) * 64 + lane]));
    }
    const float inv = 1.0f / (fmaxf(fabsf(den), num[s.vdim + 1]) + 1e-6f);
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
