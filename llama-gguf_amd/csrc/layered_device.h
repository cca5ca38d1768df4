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

// The same through inline assembly, for kernels whose LDS reads the compiler's wait-count pass does not tell apart from the DMA's
// target (transposed reads): it does not see these loads, and the kernel waits for them itself with wait_vm.
__device__ __forceinline__ void lds_dma16_untracked(const void* g, uint32_t lds_addr) {
  uint32_t keep;
  asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %2\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off\n\ts_mov_b32 m0, %0"
               : "=&s"(keep) : "v"(g), "s"(lds_addr) : "memory");
}
__device__ __forceinline__ uint32_t lds_addr_of(const void* p) {
  return (uint32_t)(uintptr_t)(const __attribute__((address_space(3))) uint8_t*)(const uint8_t*)p;
}
// all but the last n vector-memory operations have completed (n = 1 .. 20; any other n waits for all)
__device__ __forceinline__ void wait_vm(uint32_t n) {
  switch (n) {
#define LGH_WAIT_VM(N) case N: __builtin_amdgcn_s_waitcnt(0x0F70 | (N & 15) | ((N >> 4) << 14)); break;
    LGH_WAIT_VM(1) LGH_WAIT_VM(2) LGH_WAIT_VM(3) LGH_WAIT_VM(4) LGH_WAIT_VM(5) LGH_WAIT_VM(6) LGH_WAIT_VM(7) LGH_WAIT_VM(8) LGH_WAIT_VM(9)
    LGH_WAIT_VM(10) LGH_WAIT_VM(11) LGH_WAIT_VM(12) LGH_WAIT_VM(13) LGH_WAIT_VM(14) LGH_WAIT_VM(15) LGH_WAIT_VM(16) LGH_WAIT_VM(17)
    LGH_WAIT_VM(18) LGH_WAIT_VM(19) LGH_WAIT_VM(20)
#undef LGH_WAIT_VM
    default: __builtin_amdgcn_s_waitcnt(0x0F70);
  }
}

}  // namespace lgh
