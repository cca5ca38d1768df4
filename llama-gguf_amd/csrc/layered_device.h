// layered_device.h — device helpers shared by the kernels of layered.h (internal): bf16 <-> f32, the activation-type traits of the
// matrix-core fragments, block reductions, activations.
#pragma once

#include "device_utils.h"
#include "layered.h"

namespace lgh {

typedef float f32x2 __attribute__((ext_vector_type(2)));
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

__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float log_sigmoid_f(float z) { return fminf(z, 0.0f) - log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float softplus_f(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }
// a gated unit with both halves clamped (LGH_EXPERT_CLAMPED)
__device__ __forceinline__ float clamped_glu_f(float gate, float up, float limit) {
  const float g = fminf(gate, limit), u = fminf(fmaxf(up, -limit), limit);
  return g * sigmoid_f(1.702f * g) * (u + 1.0f);
}

// tanh: its odd series up to 1/4 (next term below 1e-7 of the value), beyond it 1 - 2 / (exp(2x) + 1); 1e-6 of the value everywhere
__device__ __forceinline__ float tanh_series(float x) {
  const float z = x * x;
  float s = __builtin_fmaf(z, 62.0f / 2835.0f, -17.0f / 315.0f);
  s = __builtin_fmaf(z, s, 2.0f / 15.0f);
  s = __builtin_fmaf(z, s, -1.0f / 3.0f);
  return __builtin_fmaf(x * z, s, x);
}
__device__ __forceinline__ float tanh_f(float x) {
  const float e = __builtin_amdgcn_exp2f(x * 2.8853900817779268f);
  const float far = __builtin_fmaf(-2.0f, __builtin_amdgcn_rcpf(e + 1.0f), 1.0f);
  return fabsf(x) < 0.25f ? tanh_series(x) : far;
}

// exp and sigmoid from the hardware's exp2 and reciprocal (1 ulp each, and the argument's rounding), gelu in its sigmoid form
__device__ __forceinline__ float exp_hw(float x) { return __builtin_amdgcn_exp2f(x * 1.4426950408889634f); }
__device__ __forceinline__ float sigmoid_hw(float z) { return __builtin_amdgcn_rcpf(1.0f + exp_hw(-z)); }
__device__ __forceinline__ float gelu_tanh_hw(float z) { return z * sigmoid_hw(1.5957691216057308f * __builtin_fmaf(0.044715f * z * z, z, z)); }

// what is not a number ranks last, so that every place is taken
__device__ __forceinline__ float rank_key(float z) { return z == z ? z : -INFINITY; }

// The `top` largest of E logits in LDS (padded with -inf to a multiple of 4), the first of equals first: expert e's place is the number of
// experts before it; sel[place], w[place] = its score.  One thread per expert.
__device__ __forceinline__ void rank_expert(const float* z, uint32_t E, uint32_t top, uint32_t e, int* sel, float* w) {
  const float v = z[e];
  uint32_t place = 0;
  for (uint32_t j = 0; j < E; j += 4) {
    const f32x4 q = *reinterpret_cast<const f32x4*>(z + j);
#pragma unroll
    for (uint32_t i = 0; i < 4; i++) place += q[i] > v || (q[i] == v && j + i < e) ? 1u : 0u;
  }
  if (place < top) { sel[place] = (int)e; w[place] = sigmoid_f(v); }
}

// LGH_ROUTER_SOFTMAX_GROUPS for T tokens by a whole workgroup.  z [T][ep] (LDS, ep = E rounded up to 4): logits, scores afterwards; c [T][ep],
// gm [T][groups] LDS scratch; sel, w [T][top]: the chosen ones, largest choice score first, and their weights.  Ends with a barrier.
__device__ __forceinline__ void route_groups(float* z, float* c, float* gm, uint32_t T, uint32_t E, uint32_t ep, uint32_t top, const RouteForm& f, int* sel, float* w) {
  const uint32_t tid = threadIdx.x, nt = blockDim.x, lane = tid & 63, wave = tid >> 6, nw = nt >> 6;
  for (uint32_t t = wave; t < T; t += nw) {
    float m = -INFINITY, s = 0.0f;
    for (uint32_t e = lane; e < E; e += 64) m = fmaxf(m, rank_key(z[t * ep + e]));
    m = wave_max(m);
    for (uint32_t e = lane; e < E; e += 64) { const float p = expf(rank_key(z[t * ep + e]) - m); z[t * ep + e] = p; s += p; }
    const float inv = 1.0f / wave_sum(s);
    for (uint32_t e = lane; e < ep; e += 64) {
      const float p = e < E ? z[t * ep + e] * inv : 0.0f;
      z[t * ep + e] = p;
      c[t * ep + e] = e < E ? rank_key(p + f.correction[e]) : -INFINITY;
    }
  }
  __syncthreads();
  const uint32_t gs = E / f.groups;
  for (uint32_t i = tid; i < T * f.groups; i += nt) {
    const float* p = c + i / f.groups * ep + i % f.groups * gs;
    float m = p[0];
    for (uint32_t e = 1; e < gs; e++) m = fmaxf(m, p[e]);
    gm[i] = m;
  }
  __syncthreads();
  for (uint32_t i = tid; i < T * E; i += nt) {   // (a group's members all find the same place for it)
    const uint32_t t = i / E, e = i % E, g = e / gs;
    const float* q = gm + t * f.groups;
    uint32_t place = 0;
    for (uint32_t j = 0; j < f.groups; j++) place += q[j] > q[g] || (q[j] == q[g] && j < g) ? 1u : 0u;
    if (place >= f.keep) c[t * ep + e] = -INFINITY;
  }
  __syncthreads();
  for (uint32_t i = tid; i < T * E; i += nt) {
    const uint32_t t = i / E, e = i % E;
    const float v = c[t * ep + e];
    uint32_t place = 0;
    for (uint32_t j = 0; j < E; j += 4) {
      const f32x4 q = *reinterpret_cast<const f32x4*>(c + t * ep + j);
#pragma unroll
      for (uint32_t k = 0; k < 4; k++) place += q[k] > v || (q[k] == v && j + k < e) ? 1u : 0u;
    }
    if (place < top) sel[t * top + place] = (int)e;
  }
  __syncthreads();
  for (uint32_t i = tid; i < T * top; i += nt) {
    const uint32_t t = i / top;
    float s = 0.0f;
    for (uint32_t k = 0; k < top; k++) s += z[t * ep + sel[t * top + k]];
    w[i] = z[t * ep + sel[i]] / (s + 1e-20f);
  }
  __syncthreads();
}

// ---- residual form LGH_RESIDUAL_SANDWICH_DYT, one channel ----
__device__ __forceinline__ float dyt_f(float v, float alpha, float w, float b) { return __builtin_fmaf(tanh_f(alpha * v), w, b); }

// four of the convolution's taps before position p (wave-uniform), requested but not used yet; nothing lies before position 0
struct ConvIn { float w[4], h[4]; };
__device__ __forceinline__ void conv_fetch(const ConvW& cv, uint32_t width, uint32_t c, int p, uint32_t j0, ConvIn& o) {
#pragma unroll
  for (uint32_t i = 0; i < 4; i++) {   // clamped: the loads are unconditional
    const uint32_t j = j0 + i;
    const bool ok = j < cv.taps && (int)j <= p;
    const uint32_t row = ok ? (uint32_t)(p - (int)j) % (cv.taps - 1) : 0u;
    o.w[i] = cv.w[(size_t)c * cv.taps + (ok ? cv.taps - 1 - j : 0u)];
    o.h[i] = cv.hist[(size_t)row * width + c];
  }
}
__device__ __forceinline__ float conv_use(const ConvW& cv, const ConvIn& in, int p, uint32_t j0, float s) {
#pragma unroll
  for (uint32_t i = 0; i < 4; i++) s = __builtin_fmaf(j0 + i < cv.taps && (int)(j0 + i) <= p ? in.w[i] : 0.0f, in.h[i], s);
  return s;
}
// what the residual update of a channel needs besides the sublayer's output
struct PostIn { float x, pw, pb, nw, nb, wl; ConvIn in; };
__device__ __forceinline__ void post_fetch_next(const PostUpdate& a, uint32_t c, int p, PostIn& r) {
  r.nw = a.next.w[c]; r.nb = a.next.b[c];
  if (a.conv.taps) r.wl = a.conv.w[(size_t)c * a.conv.taps + a.conv.taps - 1];
  if (a.conv.taps > 1) conv_fetch(a.conv, a.width, c, p, 1, r.in);
}
__device__ __forceinline__ void post_fetch(const PostUpdate& a, uint32_t c, int p, PostIn& r) {
  r.x = a.x[c];
  r.pw = a.post.w[c]; r.pb = a.post.b[c];
  post_fetch_next(a, c, p, r);
}
// stream value v of channel c at position p -> the next sublayer's input
__device__ __forceinline__ void post_input(const PostUpdate& a, const PostIn& r, uint32_t c, int p, float v, float nalpha) {
  const float h = dyt_f(v, nalpha, r.nw, r.nb);
  float o = h;
  if (a.conv.taps) o = __builtin_fmaf(r.wl, h, o);
  if (a.conv.taps > 1) {
    o = conv_use(a.conv, r.in, p, 1, o);
    for (uint32_t j = 5; j < a.conv.taps; j += 4) {
      ConvIn in;
      conv_fetch(a.conv, a.width, c, p, j, in);
      o = conv_use(a.conv, in, p, j, o);
    }
    a.conv.hist[(size_t)((uint32_t)p % (a.conv.taps - 1)) * a.width + c] = h;
  }
  a.hout[c] = o;
}
__device__ __forceinline__ void post_finish(const PostUpdate& a, const PostIn& r, uint32_t c, int p, float y, float palpha, float nalpha) {
  const float v = __builtin_fmaf(a.mult, dyt_f(y, palpha, r.pw, r.pb), r.x);
  a.xout[c] = v;
  post_input(a, r, c, p, v, nalpha);
}

// sum over the wave without the LDS crossbar, every lane gets it
__device__ __forceinline__ float wave_total(float v) {
  return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, wave_sum_to_lane63(v)), 63));
}

// sum over `N` neighbouring lanes, every one of them gets it
template <uint32_t N> __device__ __forceinline__ float lanes_sum(float v) {
  v += dpp_f<0xB1>(v); v += dpp_f<0x4E>(v); v += dpp_f<0x141>(v);
  if constexpr (N >= 16) v += dpp_f<0x140>(v);
  if constexpr (N >= 32) v += __shfl_xor(v, 16, 64);
  if constexpr (N >= 64) v += __shfl_xor(v, 32, 64);
  return v;
}

template <class T> __device__ __forceinline__ T to_act(float v) { return (T)v; }

// 16 bytes of a cache row as floats
template <class T, int PER> __device__ __forceinline__ void unpack_row(const u32x4& w, float* f) {
  if constexpr (sizeof(T) == 2) {
    f[0] = bf_lo(w.x); f[1] = bf_hi(w.x); f[2] = bf_lo(w.y); f[3] = bf_hi(w.y);
    f[4] = bf_lo(w.z); f[5] = bf_hi(w.z); f[6] = bf_lo(w.w); f[7] = bf_hi(w.w);
  } else {
    f[0] = __uint_as_float(w.x); f[1] = __uint_as_float(w.y); f[2] = __uint_as_float(w.z); f[3] = __uint_as_float(w.w);
  }
}

// PER values of a head's row from d0 on, 0 behind its end; vec: rows start and end at multiples of 4
template <int PER> __device__ __forceinline__ void row_chunk(const float* p, uint32_t d0, uint32_t dim, bool vec, float* o) {
  if (vec) {
#pragma unroll
    for (int i = 0; i < PER; i += 4) {
      const f32x4 v = *reinterpret_cast<const f32x4*>(p + (d0 + i < dim ? d0 + i : 0));
#pragma unroll
      for (int e = 0; e < 4; e++) o[i + e] = d0 + i < dim ? v[e] : 0.0f;
    }
  } else {
#pragma unroll
    for (int e = 0; e < PER; e++) {
      const float v = p[d0 + e < dim ? d0 + e : 0];
      o[e] = d0 + e < dim ? v : 0.0f;
    }
  }
}

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

// a wave: one head's output of a token, RMS-normed (w [vdim]) and silu-gated, times f -> o [vdim]
template <class O> __device__ __forceinline__ void head_read_out(const float* num, const float* w, const float* gate, uint32_t vdim, float eps, float f, O* o) {
  const uint32_t lane = threadIdx.x & 63;
  float ss = 0.0f;
  for (uint32_t j = lane; j < vdim; j += 64) ss = __builtin_fmaf(num[j], num[j], ss);
  const float r = f / __builtin_sqrtf(wave_sum(ss) / (float)vdim + eps);
  for (uint32_t j = lane; j < vdim; j += 64) o[j] = to_act<O>(num[j] * r * w[j] * silu_f(gate[j]));
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

// value fragment from a tile of keys (rows of `ld` elements, 16-byte chunks stored at chunk ^ (row & 7)); k slots (lane group g, j):
// bf16: keys 4g + j of the tile's first 16 rows (j < 4) and of its second 16 (j >= 4); f32: keys 4g + j of rows 16 n ..; column c0 + r16.
typedef short s16x4 __attribute__((ext_vector_type(4)));
template <class T>
__device__ __forceinline__ typename Frag<T>::V tile_value_frag(const T* tile, uint32_t ld, int n, uint32_t c0, uint32_t r16, uint32_t g) {
  if constexpr (sizeof(T) == 2) {   // lane i of a 16-lane group fetches 4 columns of key row i / 4 and receives 4 keys of column i
    const uint32_t col = c0 + (r16 & 3) * 4, row = g * 4 + (r16 >> 2);
    typedef __attribute__((address_space(3))) s16x4* lds_p;
    const T* p0 = tile + row * ld + ((col >> 3) ^ (row & 7)) * 8 + (col & 7);   // row + 16 has the same low bits
    const s16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_p)p0), b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_p)(p0 + 16 * ld));
    return __builtin_bit_cast(bf16x8, __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7));
  } else {
    const uint32_t col = c0 + r16;
    f32x4 v;
#pragma unroll
    for (uint32_t e = 0; e < 4; e++) {
      const uint32_t row = n * 16 + g * 4 + e;
      v[e] = tile[row * ld + ((col >> 2) ^ (row & 7)) * 4 + (col & 3)];
    }
    return v;
  }
}

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
