// gla.hip — gated linear attention of layered.h, all of it in 32-bit: S_t = diag(alpha_t) S_(t-1) + k_t v_t^T per head, o_t = S_t^T q_t, every
// key channel with a decay of its own, alpha = sigmoid(z)^(1 / tau).
//
// Blocks of tokens, 64 at a time.  With b_t the running sum of log alpha (in units of log2) within the chunk (b_e at its last token):
//   o_t = S_p^T (exp(b_t) q_t) + sum_(s<=t) A_ts v_s,   A_ts = sum_d q_td k_sd exp(b_td - b_sd)
//   S_e = diag(exp(b_e)) S_p + sum_s (exp(b_e - b_s) k_s) v_s^T
// The state's part is the matrix memory's chunk kernel (mlstm.hip) on queries and keys that carry their decays.  A is formed 16 x 16 tokens at a
// time: between different groups of 16 both factors are taken relative to the start of the later group, so that no exponent is positive, and
// multiplied on the f32 matrix cores; within a group exponents are differences.  Running sums are kept per group of 16 tokens.
#include "gla_device.h"

namespace lgh {

__global__ void __launch_bounds__(256) gla_step_kernel(const GlaShape s, const GlaBufs b, const int* __restrict__ pos_ptr, uint32_t pos0) {
  gla_step(s, b, pos_ptr ? (uint32_t)*pos_ptr : pos0, blockIdx.x, blockIdx.y);
}

static bool gla_ok(const GlaShape& s) {
  return s.heads && s.dim && s.vdim && s.rank && s.lds % 16 == 0 && s.lds >= s.vdim && s.ldo >= s.vdim && s.a2_ld % 8 == 0 && s.a2_ld >= s.rank && s.tau > 0.0f;
}

hipError_t gla_step_launch(const GlaShape& s, const GlaBufs& b, const int* pos_ptr, uint32_t pos0, hipStream_t st) {
  if (!gla_ok(s)) return hipErrorInvalidValue;
  hipLaunchKernelGGL(gla_step_kernel, dim3((s.vdim + 15) / 16, s.heads), dim3(256), 0, st, s, b, pos_ptr, pos0);
  return hipGetLastError();
}

constexpr uint32_t kSlab = 64, kSlabLd = kSlab + 4, kRankTile = 16;

// decays, decayed queries and keys, scores; grid (chunks, heads), 64 key channels at a time
__global__ void __launch_bounds__(256) gla_chunk_kernel(const GlaShape s, const GlaBufs b, uint32_t M) {
  __shared__ __attribute__((aligned(16))) float qs[64][kSlabLd], ks[64][kSlabLd], bs[64][kSlabLd];   // queries, keys, running log decays (per 16 tokens)
  __shared__ float tot[4][kSlab];                                                                    // a group's log decay
  __shared__ float a1s[64][kRankTile];
  const uint32_t ch = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, w = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6));
  const uint32_t r16 = lane & 15, g = lane >> 4, t0 = ch * 64, HD = s.heads * s.dim;
  const float scale = 1.0f / __builtin_sqrtf((float)s.dim), rtau = 1.4426950408889634f / s.tau;
  f32x4 acc[3];                                // scores of group w's tokens with the groups before it
  float dg[4] = {0.0f, 0.0f, 0.0f, 0.0f};      // ... within the group: query r16, keys 4g ..
#pragma unroll
  for (int j = 0; j < 3; j++) acc[j] = (f32x4)(0.0f);
  for (uint32_t d0 = 0; d0 < s.dim; d0 += kSlab) {
    const uint32_t d = d0 + lane, dc = d < s.dim ? d : s.dim - 1, row = h * s.dim + dc;
    // this thread: channel d, tokens 16 w ..
    float z[16], q[16], k[16];
#pragma unroll
    for (int i = 0; i < 16; i++) {
      const uint32_t t = t0 + w * 16 + i;
      const float* c = b.cat + (size_t)(t < M ? t : M - 1) * s.ldcat;
      q[i] = c[s.off_q + row];
      k[i] = c[s.off_k + row];
      z[i] = 0.0f;
    }
    for (uint32_t r0 = 0; r0 < s.rank; r0 += kRankTile) {
      __syncthreads();                         // (also: the slab before is used up)
      for (uint32_t i = tid; i < 64 * kRankTile; i += 256) {
        const uint32_t t = t0 + i / kRankTile, r = r0 + i % kRankTile;
        const float v = b.cat[(size_t)(t < M ? t : M - 1) * s.ldcat + s.off_a + (r < s.rank ? r : 0)];
        a1s[i / kRankTile][i % kRankTile] = r < s.rank ? v : 0.0f;
      }
      __syncthreads();
#pragma unroll
      for (uint32_t r = 0; r < kRankTile; r += 8) {
        if (r0 + r >= s.rank) break;
        float f[8];
        unpack_row<__bf16, 8>(*reinterpret_cast<const u32x4*>(b.a2 + (size_t)row * s.a2_ld + r0 + r), f);
#pragma unroll
        for (int i = 0; i < 16; i++)
#pragma unroll
          for (int e = 0; e < 8; e++) z[i] = __builtin_fmaf(f[e], a1s[w * 16 + i][r + e], z[i]);
      }
    }
    float run = 0.0f;
    const float zb = b.a2b[row];
#pragma unroll
    for (int i = 0; i < 16; i++) {
      const bool ok = t0 + w * 16 + i < M && d < s.dim;
      run += ok ? gla_log2_decay(z[i] + zb, rtau) : 0.0f;
      z[i] = run;
      q[i] = ok ? q[i] * scale : 0.0f;
      k[i] = ok ? k[i] : 0.0f;
      bs[w * 16 + i][lane] = run;
      qs[w * 16 + i][lane] = q[i];
      ks[w * 16 + i][lane] = k[i];
    }
    tot[w][lane] = run;
    __syncthreads();
    float before = 0.0f, after = 0.0f;         // the groups before and after this one
    for (uint32_t j = 0; j < 4; j++) {
      const float t = tot[j][lane];
      if (j < w) before += t;
      if (j > w) after += t;
    }
    if (d < s.dim) {
#pragma unroll
      for (int i = 0; i < 16; i++) {           // (rows behind the block's last token: zeros)
        float* o = b.qk + (size_t)(t0 + w * 16 + i) * 2 * HD + row;
        o[0] = q[i] * __builtin_amdgcn_exp2f(before + z[i]);
        o[HD] = k[i] * __builtin_amdgcn_exp2f(after + (run - z[i]));
      }
      if (w == 0) b.dec[(size_t)ch * HD + row] = __builtin_amdgcn_exp2f(run + after);
    }
    // scores with the groups before: queries relative to the start of group w
#pragma unroll
    for (uint32_t u = 0; u < kSlab; u += 16) {
      const uint32_t e0 = u + g * 4;
      f32x4 qf = *reinterpret_cast<const f32x4*>(&qs[w * 16 + r16][e0]);
      const f32x4 bq = *reinterpret_cast<const f32x4*>(&bs[w * 16 + r16][e0]);
#pragma unroll
      for (int e = 0; e < 4; e++) qf[e] *= __builtin_amdgcn_exp2f(bq[e]);
      f32x4 mid = (f32x4)(0.0f);               // groups between
#pragma unroll
      for (int j = 2; j >= 0; j--) {
        if (j >= (int)w) continue;
        f32x4 kf = *reinterpret_cast<const f32x4*>(&ks[j * 16 + r16][e0]);
        const f32x4 bk = *reinterpret_cast<const f32x4*>(&bs[j * 16 + r16][e0]), tj = *reinterpret_cast<const f32x4*>(&tot[j][e0]);
#pragma unroll
        for (int e = 0; e < 4; e++) kf[e] *= __builtin_amdgcn_exp2f(mid[e] + (tj[e] - bk[e]));
        acc[j] = Frag<float>::mma(qf, kf, acc[j]);
        mid += tj;
      }
    }
    // within the group
    for (uint32_t e0 = 0; e0 < kSlab; e0 += 4) {
      const f32x4 qv = *reinterpret_cast<const f32x4*>(&qs[w * 16 + r16][e0]), bq = *reinterpret_cast<const f32x4*>(&bs[w * 16 + r16][e0]);
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const uint32_t key = w * 16 + g * 4 + i;
        const f32x4 kv = *reinterpret_cast<const f32x4*>(&ks[key][e0]), bk = *reinterpret_cast<const f32x4*>(&bs[key][e0]);
#pragma unroll
        for (int e = 0; e < 4; e++) dg[i] = __builtin_fmaf(qv[e] * kv[e], __builtin_amdgcn_exp2f(fminf(bq[e] - bk[e], 0.0f)), dg[i]);
      }
    }
  }
  float* A = b.a + ((size_t)ch * s.heads + h) * 4096;
#pragma unroll
  for (int j = 0; j < 4; j++)
#pragma unroll
    for (int e = 0; e < 4; e++)   // the product's lane: query 4g + e, key r16
      if (j != (int)w) A[(w * 16 + g * 4 + e) * 64 + j * 16 + r16] = j < (int)w && j < 3 ? acc[j < 3 ? j : 0][e] : 0.0f;
  f32x4 v;
#pragma unroll
  for (int i = 0; i < 4; i++) v[i] = g * 4 + i <= r16 ? dg[i] : 0.0f;
  *reinterpret_cast<f32x4*>(&A[(w * 16 + r16) * 64 + w * 16 + g * 4]) = v;
}

hipError_t gla_block_launch(const GlaShape& s, const GlaBufs& b, uint32_t pos0, uint32_t M, hipStream_t st) {
  if (!gla_ok(s) || M == 0 || M > b.Mcap || b.Mcap % 64) return hipErrorInvalidValue;
  if (s.dim > kMlstmBlockDim) {   // a head's rows do not fit the state kernel's registers: token by token
    for (uint32_t t = 0; t < M; t++) {
      GlaBufs r = b;
      r.cat += (size_t)t * s.ldcat;
      r.num += (size_t)t * s.heads * s.ldo;
      if (hipError_t e = gla_step_launch(s, r, nullptr, pos0 + t, st); e != hipSuccess) return e;
    }
    return hipSuccess;
  }
  hipLaunchKernelGGL(gla_chunk_kernel, dim3((M + 63) / 64, s.heads), dim3(256), 0, st, s, b, M);
  if (hipError_t e = hipGetLastError(); e != hipSuccess) return e;
  MlstmShape ms{};
  ms.heads = s.heads; ms.dim = s.dim; ms.vdim = s.vdim; ms.lds = s.lds; ms.ldo = s.ldo;
  ms.off_k = s.heads * s.dim; ms.off_v = s.off_v; ms.ldcat = s.ldcat; ms.ldqk = 2 * s.heads * s.dim;
  MlstmBufs mb{};
  mb.cat = b.cat; mb.S = b.S; mb.num = b.num; mb.a = b.a; mb.qk = b.qk; mb.rowdec = b.dec; mb.Mcap = b.Mcap;
  return mlstm_state_launch(ms, mb, pos0, M, st);
}

template <class T>
__global__ void __launch_bounds__(256) gla_out_kernel(const GlaShape s, const GlaBufs b, T* __restrict__ out, uint32_t ldo) {
  const uint32_t t = blockIdx.x;
  for (uint32_t h = threadIdx.x >> 6; h < s.heads; h += 4)
    gla_read_out<T>(s, b.norm, b.num + ((size_t)t * s.heads + h) * s.ldo, b.cat + (size_t)t * s.ldcat, h, out + (size_t)t * ldo + (size_t)h * s.vdim);
}

hipError_t gla_out_launch(const GlaShape& s, const GlaBufs& b, uint32_t M, void* out, uint32_t ldo, bool f32, hipStream_t st) {
  if (!gla_ok(s) || M == 0) return hipErrorInvalidValue;
  if (f32) hipLaunchKernelGGL(gla_out_kernel<float>, dim3(M), dim3(256), 0, st, s, b, (float*)out, ldo);
  else hipLaunchKernelGGL(gla_out_kernel<__bf16>, dim3(M), dim3(256), 0, st, s, b, (__bf16*)out, ldo);
  return hipGetLastError();
}

}  // namespace lgh
