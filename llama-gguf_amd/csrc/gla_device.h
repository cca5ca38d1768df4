// gla_device.h — one token of gated linear attention as device functions of 256 threads (gla.hip; gated_attention.hip runs them beside its own work).
#pragma once

#include "layered_device.h"

namespace lgh {

// z of a key channel -> log2 of its decay; rtau: log2(e) / tau
__device__ __forceinline__ float gla_log2_decay(float z, float rtau) { return log_sigmoid_f(z) * rtau; }

// One token: a workgroup owns 16 columns (block cb) of head h's state, 4 lanes x 4 columns, 64 rows at a time
__device__ __forceinline__ void gla_step(const GlaShape& s, const GlaBufs& b, uint32_t pos, uint32_t cb, uint32_t h) {
  __shared__ float o_s[4][16];
  __shared__ float al[256];
  const uint32_t tid = threadIdx.x, lane = tid & 63, c4 = cb * 16 + (tid & 3) * 4, r0 = tid >> 2;
  const float* q = b.cat + s.off_q + (size_t)h * s.dim;
  const float* k = b.cat + s.off_k + (size_t)h * s.dim;
  const float* v = b.cat + s.off_v + (size_t)h * s.vdim;
  const float* a1 = b.cat + s.off_a;
  float* S = b.S + (size_t)h * s.dim * s.lds + c4;
  const float qs = 1.0f / __builtin_sqrtf((float)s.dim);
  float vv[4], o[4];
#pragma unroll
  for (int e = 0; e < 4; e++) {
    const uint32_t c = c4 + e;
    const float x = v[c < s.vdim ? c : 0];
    vv[e] = c < s.vdim ? x : 0.0f;
    o[e] = 0.0f;
  }
  for (uint32_t d0 = 0; d0 < s.dim; d0 += 256) {
    f32x4 st[4];
    float kd[4], qd[4];
#pragma unroll
    for (int i = 0; i < 4; i++) {   // (rows past the end re-read the last one and are dropped)
      const uint32_t d = d0 + i * 64 + r0, dc = d < s.dim ? d : s.dim - 1;
      st[i] = *reinterpret_cast<const f32x4*>(S + (size_t)dc * s.lds);
      kd[i] = k[dc];
      qd[i] = q[dc] * qs;
    }
    {
      const uint32_t d = d0 + tid, dc = d < s.dim ? d : s.dim - 1;
      const uint16_t* w = b.a2 + ((size_t)h * s.dim + dc) * s.a2_ld;
      float z = b.a2b[(size_t)h * s.dim + dc];
      for (uint32_t r0 = 0; r0 < s.rank; r0 += 32) {   // (rows of a2 end in zeros, the segment of a1 at a multiple of 16)
        u32x4 p[4];
        f32x4 a[8];
#pragma unroll
        for (uint32_t j = 0; j < 4; j++) {
          const uint32_t r = r0 + j * 8 < s.rank ? r0 + j * 8 : 0;
          p[j] = *reinterpret_cast<const u32x4*>(w + r);
          a[2 * j] = *reinterpret_cast<const f32x4*>(a1 + r);
          a[2 * j + 1] = *reinterpret_cast<const f32x4*>(a1 + r + 4);
        }
#pragma unroll
        for (uint32_t j = 0; j < 4; j++) {
          if (r0 + j * 8 >= s.rank) break;
          float f[8];
          unpack_row<__bf16, 8>(p[j], f);
#pragma unroll
          for (uint32_t e = 0; e < 8; e++) z = __builtin_fmaf(f[e], a[2 * j + e / 4][e & 3], z);
        }
      }
      if (d0) __syncthreads();
      al[tid] = __builtin_amdgcn_exp2f(gla_log2_decay(z, 1.4426950408889634f / s.tau));
      __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const uint32_t d = d0 + i * 64 + r0;
      if (d >= s.dim) continue;
      const float a = al[i * 64 + r0];
      f32x4 x;
#pragma unroll
      for (int e = 0; e < 4; e++) {
        x[e] = __builtin_fmaf(kd[i], vv[e], pos ? a * st[i][e] : 0.0f);   // at position 0 whatever is stored belongs to another sequence
        o[e] = __builtin_fmaf(x[e], qd[i], o[e]);
      }
      *reinterpret_cast<f32x4*>(S + (size_t)d * s.lds) = x;
    }
  }
#pragma unroll
  for (int e = 0; e < 4; e++) {   // the 16 row slots of a wave: lanes with equal lane & 3
    o[e] += __shfl_xor(o[e], 4, 64); o[e] += __shfl_xor(o[e], 8, 64); o[e] += __shfl_xor(o[e], 16, 64); o[e] += __shfl_xor(o[e], 32, 64);
    if (lane < 4) o_s[tid >> 6][lane * 4 + e] = o[e];
  }
  __syncthreads();
  if (tid < 16) {
    const uint32_t c = cb * 16 + tid;
    if (c < s.vdim) b.num[(size_t)h * s.ldo + c] = (o_s[0][tid] + o_s[1][tid]) + (o_s[2][tid] + o_s[3][tid]);
  }
}

// a wave: head h's output of one token (num, its row of cat), normed and gated -> o [vdim]
template <class O> __device__ __forceinline__ void gla_read_out(const GlaShape& s, const float* norm, const float* num, const float* cat, uint32_t h, O* o) {
  head_read_out<O>(num, norm, cat + s.off_g + (size_t)h * s.vdim, s.vdim, s.eps, s.out_scale, o);
}

}  // namespace lgh
