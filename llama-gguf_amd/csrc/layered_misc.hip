// layered_misc.hip — embedding (with the pair table), residual + layer norm, final norm of the models of layered.h.
#include "layered.h"
#include "layered_device.h"

namespace lgh {

// row of the pair table: a hash of (previous token, token); the row after the last bucket opens a sequence
__device__ __forceinline__ uint64_t bigram_row(const EmbedArgs& a, uint32_t pos, uint32_t prev, uint32_t cur) {
  if (pos == 0) return a.buckets;
  return ((uint64_t)prev * a.mul_prev + (uint64_t)cur * a.mul_cur) % a.buckets;
}

// One decode token: advances the position words, notes the token in the history, writes the residual stream.  One workgroup.
__global__ void __launch_bounds__(1024) layered_embed_kernel(const EmbedArgs a, int* state, float* __restrict__ x) {
  const int p = state[ST_NEXT];
  const uint32_t tok = (uint32_t)state[ST_TOKEN];
  const uint32_t prev = p > 0 && a.bigram ? (uint32_t)a.hist[p - 1] : 0u;
  __syncthreads();
  if (threadIdx.x == 0) {
    state[ST_POS] = p;
    state[ST_NEXT] = p + 1;
    a.hist[p] = (int)tok;
  }
  const uint16_t* e = a.embed + (size_t)tok * a.width;
  const uint16_t* b = a.bigram ? a.bigram + bigram_row(a, (uint32_t)p, prev, tok) * a.width : nullptr;
  for (uint32_t i = threadIdx.x; i < a.width; i += blockDim.x) x[i] = b ? bf_f(e[i]) + bf_f(b[i]) : bf_f(e[i]);
}

hipError_t layered_embed_launch(const EmbedArgs& a, int* state, float* x, hipStream_t st) {
  hipLaunchKernelGGL(layered_embed_kernel, dim3(1), dim3(1024), 0, st, a, state, x);
  return hipGetLastError();
}

template <class T>
__global__ void __launch_bounds__(256) layered_embed_block_kernel(const EmbedArgs a, const int* __restrict__ tokens, uint32_t pos0, float* __restrict__ x,
                                                                  T* __restrict__ xa, uint32_t ldx) {
  const uint32_t t = blockIdx.x, pos = pos0 + t;
  const uint32_t tok = (uint32_t)tokens[t];
  const uint16_t* e = a.embed + (size_t)tok * a.width;
  const uint16_t* b = nullptr;
  if (a.bigram) {
    const uint32_t prev = t ? (uint32_t)tokens[t - 1] : pos ? (uint32_t)a.hist[pos - 1] : 0u;   // this launch writes hist[pos0 ..] only
    b = a.bigram + bigram_row(a, pos, prev, tok) * a.width;
  }
  if (threadIdx.x == 0) a.hist[pos] = (int)tok;
  for (uint32_t i = threadIdx.x; i < a.width; i += 256) {
    const float v = b ? bf_f(e[i]) + bf_f(b[i]) : bf_f(e[i]);
    x[(size_t)t * a.width + i] = v;
    xa[(size_t)t * ldx + i] = to_act<T>(v);
  }
}

hipError_t layered_embed_block_launch(const EmbedArgs& a, const int* tokens, uint32_t pos0, uint32_t M, float* x, void* xa, uint32_t ldx, bool f32,
                                      hipStream_t st) {
  if (f32) hipLaunchKernelGGL(layered_embed_block_kernel<float>, dim3(M), dim3(256), 0, st, a, tokens, pos0, x, (float*)xa, ldx);
  else hipLaunchKernelGGL(layered_embed_block_kernel<__bf16>, dim3(M), dim3(256), 0, st, a, tokens, pos0, x, (__bf16*)xa, ldx);
  return hipGetLastError();
}

// layer norm (mean, then squared deviations): one workgroup per row, the row in LDS
constexpr uint32_t kNormMaxWidth = 32768;

template <class T>
__global__ void __launch_bounds__(256) resid_norm_kernel(const float* __restrict__ xin, const float* __restrict__ y, uint32_t ldy, const float* __restrict__ w,
                                                         float eps, float mult, uint32_t width, float* __restrict__ xout, T* __restrict__ xa, uint32_t ldx) {
  extern __shared__ float row[];
  __shared__ float red[16];
  const uint32_t t = blockIdx.x;
  y += (size_t)t * ldy;
  float s = 0.0f;
  for (uint32_t i = threadIdx.x; i < width; i += 256) { const float v = y[i]; row[i] = v; s += v; }
  const float mean = block_sum(s, red) / (float)width;
  float q = 0.0f;
  for (uint32_t i = threadIdx.x; i < width; i += 256) { const float d = row[i] - mean; q = __builtin_fmaf(d, d, q); }
  const float inv = 1.0f / __builtin_sqrtf(block_sum(q, red) / (float)width + eps);
  for (uint32_t i = threadIdx.x; i < width; i += 256) {
    const float v = xin[(size_t)t * width + i] + mult * ((row[i] - mean) * inv * w[i]);
    xout[(size_t)t * width + i] = v;
    if (xa) xa[(size_t)t * ldx + i] = to_act<T>(v);
  }
}

hipError_t resid_norm_launch(float* x, const float* y, uint32_t ldy, const float* w, float eps, float mult, uint32_t width, uint32_t M, void* xa,
                             uint32_t ldx, bool f32, hipStream_t st) {
  if (width > kNormMaxWidth) return hipErrorInvalidValue;
  static bool o32[64] = {}, o16[64] = {};
  const size_t lds = (size_t)width * 4;
  if (f32) {
    if (hipError_t e = lds_opt_in(reinterpret_cast<const void*>(&resid_norm_kernel<float>), kNormMaxWidth * 4, o32); e != hipSuccess) return e;
    hipLaunchKernelGGL(resid_norm_kernel<float>, dim3(M), dim3(256), lds, st, x, y, ldy, w, eps, mult, width, x, (float*)xa, ldx);
  } else {
    if (hipError_t e = lds_opt_in(reinterpret_cast<const void*>(&resid_norm_kernel<__bf16>), kNormMaxWidth * 4, o16); e != hipSuccess) return e;
    hipLaunchKernelGGL(resid_norm_kernel<__bf16>, dim3(M), dim3(256), lds, st, x, y, ldy, w, eps, mult, width, x, (__bf16*)xa, ldx);
  }
  return hipGetLastError();
}

hipError_t resid_norm_out_launch(const float* x, const float* y, const float* w, float eps, float mult, uint32_t width, float* xout, hipStream_t st) {
  if (width > kNormMaxWidth) return hipErrorInvalidValue;
  static bool opted[64] = {};
  if (hipError_t e = lds_opt_in(reinterpret_cast<const void*>(&resid_norm_kernel<float>), kNormMaxWidth * 4, opted); e != hipSuccess) return e;
  hipLaunchKernelGGL(resid_norm_kernel<float>, dim3(1), dim3(256), (size_t)width * 4, st, x, y, width, w, eps, mult, width, xout, (float*)nullptr, 0u);
  return hipGetLastError();
}

template <class T>
__global__ void __launch_bounds__(256) final_norm_rows_kernel(const float* __restrict__ x, const int* __restrict__ rows, const float* __restrict__ w, float eps,
                                                              uint32_t width, T* __restrict__ xa, uint32_t ldx) {
  __shared__ float red[16];
  const float* r = x + (size_t)rows[blockIdx.x] * width;
  float s = 0.0f;
  for (uint32_t i = threadIdx.x; i < width; i += 256) s += r[i];
  const float mean = block_sum(s, red) / (float)width;
  float q = 0.0f;
  for (uint32_t i = threadIdx.x; i < width; i += 256) { const float d = r[i] - mean; q = __builtin_fmaf(d, d, q); }
  const float inv = 1.0f / __builtin_sqrtf(block_sum(q, red) / (float)width + eps);
  for (uint32_t i = threadIdx.x; i < width; i += 256) xa[(size_t)blockIdx.x * ldx + i] = to_act<T>((r[i] - mean) * inv * w[i]);
}

hipError_t final_norm_rows_launch(const float* x, const int* rows, uint32_t n_rows, const float* w, float eps, uint32_t width, void* xa, uint32_t ldx,
                                  bool f32, hipStream_t st) {
  if (f32) hipLaunchKernelGGL(final_norm_rows_kernel<float>, dim3(n_rows), dim3(256), 0, st, x, rows, w, eps, width, (float*)xa, ldx);
  else hipLaunchKernelGGL(final_norm_rows_kernel<__bf16>, dim3(n_rows), dim3(256), 0, st, x, rows, w, eps, width, (__bf16*)xa, ldx);
  return hipGetLastError();
}

}  // namespace lgh
