// layered_device.h — device helpers shared by the kernels of layered.h (internal): bf16 <-> f32, the activation-type traits of the
// matrix-core fragments, block reductions, activations.
#pragma once

#include "device_utils.h"

namespace lgh {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float bf_lo(uint32_t w) { return __uint_as_float(w << 16); }
__device__ __forceinline__ float bf_hi(uint32_t w) { return __uint_as_float(w & 0xFFFF0000u); }
__device__ __forceinline__ float bf_f(uint16_t w) { return __uint_as_float((uint32_t)w << 16); }

// the tanh form of gelu
__device__ __forceinline__ float gelu_tanh_f(float z) {
  const float inner = 0.7978845608028654f * (z + 0.044715f * z * z * z);
  return 0.5f * z * (1.0f + tanhf(inner));
}
__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }

// sum over a workgroup of up to 16 waves; every thread gets the result.  red: 16 floats of LDS, free again after the call.
__device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_sum(v);
  const uint32_t nw = (blockDim.x + 63) >> 6;
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float t = 0.0f;
  for (uint32_t i = 0; i < nw; i++) t += red[i];
  __syncthreads();
  return t;
}

// A matrix-core "unit": 16 bytes of the k axis per lane.  bf16: one v_mfma_f32_16x16x32_bf16 over 32 k (lane group g holds k = 8g ..
// 8g + 7).  f32: four v_mfma_f32_16x16x4_f32 over 16 k, the j-th one over k = {j, 4 + j, 8 + j, 12 + j} (lane group g holds
// k = 4g .. 4g + 3).  Both operands use the same assignment, so the sum runs over every k once.
template <class T> struct Frag;
template <> struct Frag<__bf16> {
  static constexpr int KU = 32, PER = 8;
  typedef bf16x8 V;
  static __device__ __forceinline__ V zero() { V v; for (int i = 0; i < 8; i++) v[i] = (__bf16)0.0f; return v; }
  static __device__ __forceinline__ V load(const __bf16* p) { return *reinterpret_cast<const V*>(p); }
  static __device__ __forceinline__ f32x4 mma(V a, V b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }
};
template <> struct Frag<float> {
  static constexpr int KU = 16, PER = 4;
  typedef f32x4 V;
  static __device__ __forceinline__ V zero() { return (f32x4)(0.0f); }
  static __device__ __forceinline__ V load(const float* p) { return *reinterpret_cast<const V*>(p); }
  static __device__ __forceinline__ f32x4 mma(V a, V b, f32x4 c) {
#pragma unroll
    for (int j = 0; j < 4; j++) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[j], b[j], c, 0, 0, 0);
    return c;
  }
};

template <class T> __device__ __forceinline__ T to_act(float v) { return (T)v; }

// 16 bytes per lane from global memory straight into LDS; lane l's bytes land at lds + 16 l (lds: wave-uniform)
__device__ __forceinline__ void lds_dma16(const void* g, void* lds) {
  __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)g, (__attribute__((address_space(3))) void*)lds, 16, 0, 0);
}

}  // namespace lgh
