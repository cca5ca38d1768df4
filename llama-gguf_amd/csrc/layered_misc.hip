// layered_misc.hip — embedding (with the pair table), residual updates of all forms (layer norm; squashing norms with a short
// convolution; RMS norm in front of a sublayer), final norm of the models of layered.h.
#include "layered.h"
#include "layered_device.h"

namespace lgh {

// row of the pair table: a hash of (previous token, token); the row after the last bucket opens a sequence
__device__ __forceinline__ uint64_t bigram_row(const EmbedArgs& a, uint32_t pos, uint32_t prev, uint32_t cur) {
  if (pos == 0) return a.buckets;
  return ((uint64_t)prev * a.mul_prev + (uint64_t)cur * a.mul_cur) % a.buckets;
}

// One decode token: advances the position words, notes the token in the history, writes the residual stream (and, with `post`, the first
// sublayer's input).  One workgroup.
__global__ void __launch_bounds__(1024) layered_embed_kernel(const EmbedArgs a, int* state, float* __restrict__ x, const PostUpdate post, int with_post) {
  const int p = __builtin_amdgcn_readfirstlane(state[ST_NEXT]);
  const uint32_t tok = (uint32_t)__builtin_amdgcn_readfirstlane(state[ST_TOKEN]);
  const uint32_t prev = p > 0 && a.bigram ? (uint32_t)a.hist[p - 1] : 0u;
  __syncthreads();
  if (threadIdx.x == 0) {
    state[ST_POS] = p;
    state[ST_NEXT] = p + 1;
    a.hist[p] = (int)tok;
  }
  const uint16_t* e = a.embed + (size_t)tok * a.ld;
  const uint16_t* b = a.bigram ? a.bigram + bigram_row(a, (uint32_t)p, prev, tok) * a.width : nullptr;
  const float alpha = with_post ? *post.next.alpha : 0.0f;
  constexpr uint32_t U = 4;   // channels a thread has in flight
  for (uint32_t i0 = threadIdx.x; i0 < a.width; i0 += U * 1024) {
    PostIn r[U];
    float v[U];
#pragma unroll
    for (uint32_t u = 0; u < U; u++) {
      const uint32_t i = i0 + u * 1024 < a.width ? i0 + u * 1024 : i0;
      v[u] = b ? bf_f(e[i]) + bf_f(b[i]) : bf_f(e[i]);
      if (with_post) post_fetch_next(post, i, p, r[u]);
    }
#pragma unroll
    for (uint32_t u = 0; u < U; u++) {
      const uint32_t i = i0 + u * 1024;
      if (i >= a.width) break;
      x[i] = v[u];
      if (with_post) post_input(post, r[u], i, p, v[u], alpha);
    }
  }
}

hipError_t layered_embed_launch(const EmbedArgs& a, int* state, float* x, const PostUpdate* post, hipStream_t st) {
  if (post && (post->width != a.width || !post->hout || !post->next.w || !post->next.b || !post->next.alpha)) return hipErrorInvalidValue;
  hipLaunchKernelGGL(layered_embed_kernel, dim3(1), dim3(1024), 0, st, a, state, x, post ? *post : PostUpdate(), post ? 1 : 0);
  return hipGetLastError();
}

template <class T>
__global__ void __launch_bounds__(256) layered_embed_block_kernel(const EmbedArgs a, const int* __restrict__ tokens, uint32_t pos0, float* __restrict__ x,
                                                                  T* __restrict__ xa, uint32_t ldx) {
  const uint32_t t = blockIdx.x, pos = pos0 + t;
  const uint32_t tok = (uint32_t)tokens[t];
  const uint16_t* e = a.embed + (size_t)tok * a.ld;
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

template <class T>
__global__ void __launch_bounds__(256) final_dyt_rows_kernel(const float* __restrict__ x, const int* __restrict__ rows, const DytW n, uint32_t width, T* __restrict__ xa,
                                                             uint32_t ldx) {
  const float* r = x + (size_t)rows[blockIdx.x] * width;
  const float alpha = *n.alpha;
  for (uint32_t i = threadIdx.x; i < width; i += 256) xa[(size_t)blockIdx.x * ldx + i] = to_act<T>(dyt_f(r[i], alpha, n.w[i], n.b[i]));
}

hipError_t final_dyt_rows_launch(const float* x, const int* rows, uint32_t n_rows, const DytW& n, uint32_t width, void* xa, uint32_t ldx, bool f32, hipStream_t st) {
  if (f32) hipLaunchKernelGGL(final_dyt_rows_kernel<float>, dim3(n_rows), dim3(256), 0, st, x, rows, n, width, (float*)xa, ldx);
  else hipLaunchKernelGGL(final_dyt_rows_kernel<__bf16>, dim3(n_rows), dim3(256), 0, st, x, rows, n, width, (__bf16*)xa, ldx);
  return hipGetLastError();
}

template <class T>
__global__ void __launch_bounds__(256) final_rms_rows_kernel(const float* __restrict__ x, const int* __restrict__ rows, const float* __restrict__ w, float eps, float scale,
                                                             uint32_t width, T* __restrict__ xa, uint32_t ldx) {
  __shared__ float red[16];
  const float* r = x + (size_t)rows[blockIdx.x] * width;
  float q = 0.0f;
  for (uint32_t i = threadIdx.x; i < width; i += 256) q = __builtin_fmaf(r[i], r[i], q);
  const float inv = 1.0f / __builtin_sqrtf(block_sum(q, red) / (float)width + eps) * scale;
  for (uint32_t i = threadIdx.x; i < width; i += 256) xa[(size_t)blockIdx.x * ldx + i] = to_act<T>(r[i] * inv * (1.0f + w[i]));
}

hipError_t final_rms_rows_launch(const float* x, const int* rows, uint32_t n_rows, const float* w, float eps, float scale, uint32_t width, void* xa, uint32_t ldx,
                                 bool f32, hipStream_t st) {
  if (f32) hipLaunchKernelGGL(final_rms_rows_kernel<float>, dim3(n_rows), dim3(256), 0, st, x, rows, w, eps, scale, width, (float*)xa, ldx);
  else hipLaunchKernelGGL(final_rms_rows_kernel<__bf16>, dim3(n_rows), dim3(256), 0, st, x, rows, w, eps, scale, width, (__bf16*)xa, ldx);
  return hipGetLastError();
}

__global__ void __launch_bounds__(256) resid_add_kernel(const float* __restrict__ x, const float* __restrict__ y, float mult, uint32_t width, float* __restrict__ xout) {
  const uint32_t i = blockIdx.x * 256 + threadIdx.x;
  if (i < width) xout[i] = __builtin_fmaf(mult, y[i], x[i]);
}

hipError_t resid_add_launch(const float* x, const float* y, float mult, uint32_t width, float* xout, hipStream_t st) {
  hipLaunchKernelGGL(resid_add_kernel, dim3((width + 255) / 256), dim3(256), 0, st, x, y, mult, width, xout);
  return hipGetLastError();
}

// ------------------------------------------------------------------------------------------------
// LGH_RESIDUAL_SANDWICH_DYT over a block.  A wave = 64 * V channels of kDytTokens tokens, walked in order; the convolution's inputs of the
// last taps positions lie in LDS, every thread its own channels (no barriers).  The taps - 1 tokens before a wave's first are formed again
// from the stream before the update, the ones before the block come from the history.
// ------------------------------------------------------------------------------------------------
constexpr int kDytTokens = 16;

template <int V> struct VecF { float v[V]; };
template <int V> __device__ __forceinline__ VecF<V> load_vec(const float* p) {
  VecF<V> r;
  if constexpr (V == 4) { const f32x4 q = *reinterpret_cast<const f32x4*>(p); r.v[0] = q.x; r.v[1] = q.y; r.v[2] = q.z; r.v[3] = q.w; }
  else if constexpr (V == 2) { const f32x2 q = *reinterpret_cast<const f32x2*>(p); r.v[0] = q.x; r.v[1] = q.y; }
  else r.v[0] = p[0];
  return r;
}
template <int V> __device__ __forceinline__ void store_vec(float* p, const VecF<V>& a) {
  if constexpr (V == 4) { f32x4 q; q.x = a.v[0]; q.y = a.v[1]; q.z = a.v[2]; q.w = a.v[3]; *reinterpret_cast<f32x4*>(p) = q; }
  else if constexpr (V == 2) { f32x2 q; q.x = a.v[0]; q.y = a.v[1]; *reinterpret_cast<f32x2*>(p) = q; }
  else p[0] = a.v[0];
}

// y of one token's channels: the sublayer's output plus its experts' rows
template <int V> __device__ __forceinline__ VecF<V> add_pairs(VecF<V> y, const float* pairs, uint32_t ldp, const int* slot, uint32_t top, uint32_t c) {
  for (uint32_t s = 0; s < top; s += 4) {   // four rows in flight
    VecF<V> p[4];
#pragma unroll
    for (uint32_t k = 0; k < 4; k++) p[k] = load_vec<V>(pairs + (size_t)slot[s + k < top ? s + k : s] * ldp + c);
#pragma unroll
    for (uint32_t k = 0; k < 4; k++)
      if (s + k < top)
#pragma unroll
        for (int i = 0; i < V; i++) y.v[i] += p[k].v[i];
  }
  return y;
}

template <class T, int V>
__global__ void __launch_bounds__(256) dyt_block_kernel(const DytBlock a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];   // [taps][256][V] inputs, [taps][256][V] filters
  const uint32_t tid = threadIdx.x, lane = tid & 63, c0 = (blockIdx.x * 64 + lane) * V;
  const int t0 = (int)((blockIdx.y * 4 + (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6))) * kDytTokens);
  if (t0 >= (int)a.M) return;
  const int t1 = t0 + kDytTokens < (int)a.M ? t0 + kDytTokens : (int)a.M;
  const bool live = c0 < a.width;
  const uint32_t c = live ? c0 : 0, W = a.width;
  const int taps = (int)a.conv.taps, back = taps ? taps - 1 : 0;
  const bool upd = a.xout != nullptr, nxt = a.xa != nullptr;
  float* ring = lds + tid * V;
  float* filt = ring + (size_t)taps * 256 * V;
  for (int j = 0; j < taps; j++)
#pragma unroll
    for (int i = 0; i < V; i++) filt[j * 256 * V + i] = a.conv.w[(size_t)(c + i) * taps + j];
  VecF<V> pw, pb, nw, nb;
  float pal = 0.0f, nal = 0.0f;
  if (upd) { pw = load_vec<V>(a.post.w + c); pb = load_vec<V>(a.post.b + c); pal = *a.post.alpha; }
  if (nxt) { nw = load_vec<V>(a.next.w + c); nb = load_vec<V>(a.next.b + c); nal = *a.next.alpha; }
  // a group of tokens requested while the one before it is worked on: the stream, the sublayer's output, its first two experts' rows
  constexpr int G = 4, P = 2;
  struct Group { VecF<V> x[G], y[G], p[G][P]; };
  const int n_pairs = upd && a.pairs ? (int)a.top : 0;
  auto request = [&](int t, Group& o) {
#pragma unroll
    for (int g = 0; g < G; g++) {
      const size_t tc = (size_t)(t + g < 0 ? 0 : t + g < t1 ? t + g : t1 - 1);
      o.x[g] = load_vec<V>(a.x + tc * W + c);
      if (upd && a.y) o.y[g] = load_vec<V>(a.y + tc * a.ldy + c);
#pragma unroll
      for (int k = 0; k < P; k++)
        if (k < n_pairs) o.p[g][k] = load_vec<V>(a.pairs + (size_t)a.slot[tc * a.top + k] * a.ldp + c);
    }
  };
  const int first = nxt ? t0 - back : t0;
  Group nx;
  request(first, nx);
  int at = 0;                                       // ring row of token t
  for (int tg = first; tg < t1; tg += G) {
    const Group cu = nx;
    if (tg + G < t1) request(tg + G, nx);
#pragma unroll
    for (int g = 0; g < G; g++) {
      const int t = tg + g;
      if (t >= t1) break;
      VecF<V> v = cu.x[g], h, y;
      if (t < 0) {                                    // before the block
        const int p = (int)a.pos0 + t;
#pragma unroll
        for (int i = 0; i < V; i++) h.v[i] = 0.0f;
        if (p >= 0) h = load_vec<V>(a.conv.hist + (size_t)(p % back) * W + c);
      } else {
        if (upd) {
#pragma unroll
          for (int i = 0; i < V; i++) y.v[i] = a.y ? cu.y[g].v[i] : 0.0f;
#pragma unroll
          for (int k = 0; k < P; k++)
            if (k < n_pairs)
#pragma unroll
              for (int i = 0; i < V; i++) y.v[i] += cu.p[g][k].v[i];
          if (n_pairs > P) y = add_pairs<V>(y, a.pairs, a.ldp, a.slot + (size_t)t * a.top + P, a.top - P, c);
#pragma unroll
          for (int i = 0; i < V; i++) v.v[i] = __builtin_fmaf(a.mult, dyt_f(y.v[i], pal, pw.v[i], pb.v[i]), v.v[i]);
          if (t >= t0 && live) store_vec<V>(a.xout + (size_t)t * W + c, v);
        }
        if (!nxt) continue;
#pragma unroll
        for (int i = 0; i < V; i++) h.v[i] = dyt_f(v.v[i], nal, nw.v[i], nb.v[i]);
      }
      if (taps) store_vec<V>(ring + at * 256 * V, h);
      if (t >= t0) {
        VecF<V> o = h;
        int r = at + 1 < taps ? at + 1 : 0;           // the oldest input
        for (int j = 0; j < taps; j++) {
          const VecF<V> q = load_vec<V>(ring + r * 256 * V), w = load_vec<V>(filt + j * 256 * V);
#pragma unroll
          for (int i = 0; i < V; i++) o.v[i] = __builtin_fmaf(w.v[i], q.v[i], o.v[i]);
          r = r + 1 < taps ? r + 1 : 0;
        }
        if (live) {
          T* dst = reinterpret_cast<T*>(a.xa) + (size_t)t * a.ldx + c;
          T q[V];
#pragma unroll
          for (int i = 0; i < V; i++) q[i] = to_act<T>(o.v[i]);
          __builtin_memcpy(__builtin_assume_aligned(dst, sizeof(q)), q, sizeof(q));
          if (t >= (int)a.M - back) store_vec<V>(a.tail + (size_t)((int)a.M - 1 - t) * W + c, h);
        }
      }
      at = at + 1 < taps ? at + 1 : 0;
    }
  }
}

template <class T, int V>
static hipError_t dyt_block_go(const DytBlock& a, hipStream_t st) {
  static bool opted[64] = {};
  const size_t lds = (size_t)a.conv.taps * 2 * 256 * V * 4;
  if (lds > 156 * 1024) return hipErrorInvalidValue;
  if (hipError_t e = lds_opt_in(reinterpret_cast<const void*>(&dyt_block_kernel<T, V>), 156 * 1024, opted); e != hipSuccess) return e;
  hipLaunchKernelGGL((dyt_block_kernel<T, V>), dim3((a.width + 64 * V - 1) / (64 * V), (a.M + 4 * kDytTokens - 1) / (4 * kDytTokens)), dim3(256), lds, st, a);
  return hipGetLastError();
}

hipError_t dyt_block_launch(const DytBlock& a, bool f32, hipStream_t st) {
  const bool upd = a.xout != nullptr, nxt = a.xa != nullptr;
  if (!a.x || a.M == 0 || (!upd && !nxt) || a.xout == a.x || (upd && (!(a.y || a.pairs) || !a.post.w || !a.post.b || !a.post.alpha)) ||
      (a.pairs && !a.slot) || (nxt && (!a.next.w || !a.next.b || !a.next.alpha || a.ldx < a.width)) || (a.conv.taps && !a.conv.w) ||
      (a.conv.taps > 1 && (!a.conv.hist || !a.tail)) || (!nxt && a.conv.taps))
    return hipErrorInvalidValue;
  const bool even = a.width % 4 == 0 && (!a.y || a.ldy % 4 == 0) && (!a.pairs || a.ldp % 4 == 0) && (!nxt || a.ldx % 4 == 0) && a.conv.taps <= 16;
  if (even && (uint64_t)a.width * a.M <= 1u << 24) return f32 ? dyt_block_go<float, 2>(a, st) : dyt_block_go<__bf16, 2>(a, st);   // (enough waves)
  if (even) return f32 ? dyt_block_go<float, 4>(a, st) : dyt_block_go<__bf16, 4>(a, st);
  return f32 ? dyt_block_go<float, 1>(a, st) : dyt_block_go<__bf16, 1>(a, st);
}

// ------------------------------------------------------------------------------------------------
// LGH_RESIDUAL_PRE_RMS over a block: a workgroup per token, the new stream row in LDS between the sum of its squares and its use
// ------------------------------------------------------------------------------------------------
template <class T, int V>
__global__ void __launch_bounds__(256) pre_block_kernel(const PreBlock a) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[16];
  const uint32_t t = blockIdx.x;
  float* x = a.x + (size_t)t * a.width;
  T* xa = reinterpret_cast<T*>(a.xa) + (size_t)t * a.ldx;
  const int* slot = a.slot + (size_t)t * a.top;
  float q = 0.0f, id_w = 0.0f;
  if (a.pairs)
    for (uint32_t s = 0; s < a.top; s++) id_w += slot[s] < 0 ? a.selw[(size_t)t * a.top + s] : 0.0f;
  for (uint32_t c = threadIdx.x * V; c < a.width; c += 256 * V) {
    VecF<V> v = load_vec<V>(x + c), y;
#pragma unroll
    for (int i = 0; i < V; i++) y.v[i] = 0.0f;
    if (a.y) y = load_vec<V>(a.y + (size_t)t * a.ldy + c);
    if (a.pairs) {
      for (uint32_t s = 0; s < a.top; s += 4) {   // four rows in flight
        VecF<V> p[4];
        float f[4];
#pragma unroll
        for (uint32_t k = 0; k < 4; k++) {
          const int r = slot[s + k < a.top ? s + k : s];
          f[k] = s + k < a.top && r >= 0 ? 1.0f : 0.0f;
          p[k] = load_vec<V>(a.pairs + (size_t)(r >= 0 ? r : 0) * a.ldp + c);
        }
#pragma unroll
        for (uint32_t k = 0; k < 4; k++)
          if (f[k] != 0.0f)
#pragma unroll
            for (int i = 0; i < V; i++) y.v[i] += p[k].v[i];
      }
      if (id_w != 0.0f)
#pragma unroll
        for (int i = 0; i < V; i++) y.v[i] = __builtin_fmaf(id_w, (float)xa[c + i], y.v[i]);
    }
#pragma unroll
    for (int i = 0; i < V; i++) {
      v.v[i] = __builtin_fmaf(a.mult, y.v[i], v.v[i]);
      q = __builtin_fmaf(v.v[i], v.v[i], q);
    }
    store_vec<V>(row + c, v);
    if (a.y || a.pairs) store_vec<V>(x + c, v);
  }
  if (!a.nw) return;
  const float inv = 1.0f / __builtin_sqrtf(block_sum(q, red) / (float)a.width + a.eps);
  for (uint32_t c = threadIdx.x * V; c < a.width; c += 256 * V) {   // (every thread its own channels again)
    const VecF<V> v = load_vec<V>(row + c), w = load_vec<V>(a.nw + c);
    T o[V];
#pragma unroll
    for (int i = 0; i < V; i++) o[i] = to_act<T>(v.v[i] * inv * (1.0f + w.v[i]));
    __builtin_memcpy(__builtin_assume_aligned(xa + c, sizeof(o)), o, sizeof(o));
  }
}

template <class T, int V>
static hipError_t pre_block_go(const PreBlock& a, hipStream_t st) {
  static bool opted[64] = {};
  if (hipError_t e = lds_opt_in(reinterpret_cast<const void*>(&pre_block_kernel<T, V>), kNormMaxWidth * 4, opted); e != hipSuccess) return e;
  hipLaunchKernelGGL((pre_block_kernel<T, V>), dim3(a.M), dim3(256), (size_t)a.width * 4, st, a);
  return hipGetLastError();
}

hipError_t pre_block_launch(const PreBlock& a, bool f32, hipStream_t st) {
  if (!a.x || !a.xa || a.M == 0 || a.width == 0 || a.width > kNormMaxWidth || a.ldx < a.width || (a.pairs && (!a.slot || !a.selw || a.top == 0))) return hipErrorInvalidValue;
  const bool v4 = a.width % 4 == 0 && (!a.y || a.ldy % 4 == 0) && (!a.pairs || a.ldp % 4 == 0) && a.ldx % 4 == 0;
  if (v4) return f32 ? pre_block_go<float, 4>(a, st) : pre_block_go<__bf16, 4>(a, st);
  return f32 ? pre_block_go<float, 1>(a, st) : pre_block_go<__bf16, 1>(a, st);
}

// ------------------------------------------------------------------------------------------------
// LGH_RESIDUAL_SANDWICH_LN over a block: a workgroup per token, the row in LDS (every thread its own channels)
// ------------------------------------------------------------------------------------------------
template <int V> __device__ __forceinline__ void ln_stats(const float* row, uint32_t width, float eps, float* red, float& mean, float& inv) {
  float s = 0.0f, q = 0.0f;
  for (uint32_t c = threadIdx.x * V; c < width; c += 256 * V) {
    const VecF<V> v = load_vec<V>(row + c);
#pragma unroll
    for (int i = 0; i < V; i++) s += v.v[i];
  }
  mean = block_sum(s, red) / (float)width;
  for (uint32_t c = threadIdx.x * V; c < width; c += 256 * V) {
    const VecF<V> v = load_vec<V>(row + c);
#pragma unroll
    for (int i = 0; i < V; i++) { const float d = v.v[i] - mean; q = __builtin_fmaf(d, d, q); }
  }
  inv = 1.0f / __builtin_sqrtf(block_sum(q, red) / (float)width + eps);
}

template <class T, int V>
__global__ void __launch_bounds__(256) ln_block_kernel(const LnBlock a) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[16];
  const uint32_t t = blockIdx.x;
  float* x = a.x + (size_t)t * a.width;
  float mean, inv;
  if (a.y) {
    const float* y = a.y + (size_t)t * a.ldy;
    for (uint32_t c = threadIdx.x * V; c < a.width; c += 256 * V) store_vec<V>(row + c, load_vec<V>(y + c));
    ln_stats<V>(row, a.width, a.eps, red, mean, inv);
    for (uint32_t c = threadIdx.x * V; c < a.width; c += 256 * V) {
      VecF<V> v = load_vec<V>(x + c);
      const VecF<V> z = load_vec<V>(row + c), w = load_vec<V>(a.pw + c);
#pragma unroll
      for (int i = 0; i < V; i++) v.v[i] = __builtin_fmaf(a.mult, (z.v[i] - mean) * inv * w.v[i], v.v[i]);
      store_vec<V>(row + c, v);
      store_vec<V>(x + c, v);
    }
  } else {
    for (uint32_t c = threadIdx.x * V; c < a.width; c += 256 * V) store_vec<V>(row + c, load_vec<V>(x + c));
  }
  if (!a.nw) return;
  ln_stats<V>(row, a.width, a.eps, red, mean, inv);
  T* xa = reinterpret_cast<T*>(a.xa) + (size_t)t * a.ldx;
  for (uint32_t c = threadIdx.x * V; c < a.width; c += 256 * V) {
    const VecF<V> v = load_vec<V>(row + c), w = load_vec<V>(a.nw + c);
    T o[V];
#pragma unroll
    for (int i = 0; i < V; i++) o[i] = to_act<T>((v.v[i] - mean) * inv * w.v[i]);
    __builtin_memcpy(__builtin_assume_aligned(xa + c, sizeof(o)), o, sizeof(o));
  }
}

template <class T, int V>
static hipError_t ln_block_go(const LnBlock& a, hipStream_t st) {
  static bool opted[64] = {};
  if (hipError_t e = lds_opt_in(reinterpret_cast<const void*>(&ln_block_kernel<T, V>), kNormMaxWidth * 4, opted); e != hipSuccess) return e;
  hipLaunchKernelGGL((ln_block_kernel<T, V>), dim3(a.M), dim3(256), (size_t)a.width * 4, st, a);
  return hipGetLastError();
}

hipError_t ln_block_launch(const LnBlock& a, bool f32, hipStream_t st) {
  if (!a.x || a.M == 0 || a.width == 0 || a.width > kNormMaxWidth || (a.y && (!a.pw || a.ldy < a.width)) || (a.nw && (!a.xa || a.ldx < a.width)) || (!a.y && !a.nw)) return hipErrorInvalidValue;
  const bool v4 = a.width % 4 == 0 && (!a.y || a.ldy % 4 == 0) && a.ldx % 4 == 0;
  if (v4) return f32 ? ln_block_go<float, 4>(a, st) : ln_block_go<__bf16, 4>(a, st);
  return f32 ? ln_block_go<float, 1>(a, st) : ln_block_go<__bf16, 1>(a, st);
}

// a wave per row, V values at a time
template <class T, int V>
__global__ void __launch_bounds__(256) rms_cols_kernel(const float* __restrict__ x, uint32_t ld, const float* __restrict__ w, float eps, uint32_t n, uint32_t M, T* __restrict__ xa,
                                                       uint32_t ldx) {
  const uint32_t t = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (t >= M) return;
  const float* r = x + (size_t)t * ld;
  T* o = xa + (size_t)t * ldx;
  constexpr uint32_t U = 8, S = 64 * V;   // loads of a lane kept between the two passes
  VecF<V> v[U];
  float q = 0.0f;
#pragma unroll
  for (uint32_t u = 0; u < U; u++) {
    const uint32_t c = lane * V + u * S;
    v[u] = load_vec<V>(r + (c < n ? c : 0));
#pragma unroll
    for (int i = 0; i < V; i++) q = c < n ? __builtin_fmaf(v[u].v[i], v[u].v[i], q) : q;
  }
  for (uint32_t c = lane * V + U * S; c < n; c += S) {
    const VecF<V> z = load_vec<V>(r + c);
#pragma unroll
    for (int i = 0; i < V; i++) q = __builtin_fmaf(z.v[i], z.v[i], q);
  }
  const float inv = 1.0f / __builtin_sqrtf(wave_sum(q) / (float)n + eps);
  auto put = [&](uint32_t c, const VecF<V>& z) {
    const VecF<V> wt = load_vec<V>(w + c);
    T d[V];
#pragma unroll
    for (int i = 0; i < V; i++) d[i] = to_act<T>(z.v[i] * inv * wt.v[i]);
    __builtin_memcpy(__builtin_assume_aligned(o + c, sizeof(d)), d, sizeof(d));
  };
#pragma unroll
  for (uint32_t u = 0; u < U; u++)
    if (lane * V + u * S < n) put(lane * V + u * S, v[u]);
  for (uint32_t c = lane * V + U * S; c < n; c += S) put(c, load_vec<V>(r + c));
}

hipError_t rms_cols_launch(const float* x, uint32_t ld, const float* w, float eps, uint32_t n, uint32_t M, void* xa, uint32_t ldx, bool f32, hipStream_t st) {
  if (!x || !w || !xa || n == 0 || M == 0 || ldx < n || ld < n) return hipErrorInvalidValue;
  const dim3 grid((M + 3) / 4), th(256);
  const bool v4 = n % 4 == 0 && ld % 4 == 0 && ldx % 4 == 0 && (uintptr_t)x % 16 == 0;
  if (f32 && v4) hipLaunchKernelGGL((rms_cols_kernel<float, 4>), grid, th, 0, st, x, ld, w, eps, n, M, (float*)xa, ldx);
  else if (f32) hipLaunchKernelGGL((rms_cols_kernel<float, 1>), grid, th, 0, st, x, ld, w, eps, n, M, (float*)xa, ldx);
  else if (v4) hipLaunchKernelGGL((rms_cols_kernel<__bf16, 4>), grid, th, 0, st, x, ld, w, eps, n, M, (__bf16*)xa, ldx);
  else hipLaunchKernelGGL((rms_cols_kernel<__bf16, 1>), grid, th, 0, st, x, ld, w, eps, n, M, (__bf16*)xa, ldx);
  return hipGetLastError();
}

__global__ void __launch_bounds__(256) vec_mul_kernel(float* __restrict__ x, const float* __restrict__ y, uint32_t n) {
  const uint32_t i = blockIdx.x * 256 + threadIdx.x;
  if (i < n) x[i] *= y[i];
}

hipError_t vec_mul_launch(float* x, const float* y, uint32_t n, hipStream_t st) {
  hipLaunchKernelGGL(vec_mul_kernel, dim3((n + 255) / 256), dim3(256), 0, st, x, y, n);
  return hipGetLastError();
}

__global__ void __launch_bounds__(256) conv_store_kernel(const float* __restrict__ tails, float* __restrict__ hists, uint32_t back, uint32_t width, uint32_t last) {
  const uint32_t c = blockIdx.x * 256 + threadIdx.x, i = blockIdx.y, k = blockIdx.z;
  if (c < width) hists[((size_t)k * back + (last - i) % back) * width + c] = tails[((size_t)k * back + i) * width + c];
}

hipError_t conv_store_launch(const float* tails, float* hists, uint32_t n_sub, uint32_t taps, uint32_t width, uint32_t pos0, uint32_t M, hipStream_t st) {
  if (taps < 2 || M == 0) return hipErrorInvalidValue;
  const uint32_t back = taps - 1;
  hipLaunchKernelGGL(conv_store_kernel, dim3((width + 255) / 256, M < back ? M : back, n_sub), dim3(256), 0, st, tails, hists, back, width, pos0 + M - 1);
  return hipGetLastError();
}

__global__ void __launch_bounds__(256) pair_sum_kernel(float* __restrict__ y, uint32_t ldy, const float* __restrict__ pairs, uint32_t ldp, const int* __restrict__ slot,
                                                       uint32_t top, uint32_t width, int add) {
  const uint32_t t = blockIdx.x;
  for (uint32_t c = threadIdx.x; c < width; c += 256) {
    VecF<1> v;
    v.v[0] = add ? y[(size_t)t * ldy + c] : 0.0f;
    y[(size_t)t * ldy + c] = add_pairs<1>(v, pairs, ldp, slot + (size_t)t * top, top, c).v[0];
  }
}

hipError_t pair_sum_launch(float* y, uint32_t ldy, const float* pairs, uint32_t ldp, const int* slot, uint32_t top, uint32_t width, uint32_t M, bool add, hipStream_t st) {
  if (!y || !pairs || !slot || M == 0) return hipErrorInvalidValue;
  hipLaunchKernelGGL(pair_sum_kernel, dim3(M), dim3(256), 0, st, y, ldy, pairs, ldp, slot, top, width, add ? 1 : 0);
  return hipGetLastError();
}

}  // namespace lgh
