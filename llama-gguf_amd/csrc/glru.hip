// glru.hip — the gated linear recurrence of layered.h.  Beside a gelu branch y, per channel: u = conv(x) + bias over the last `taps` positions;
// r = sigmoid(R u + b), i = sigmoid(I u + b) with block-diagonal R, I; log a = -8 r softplus(lam); S_t = a S_(t-1) + sqrt(1 - a^2) i u; out S * y.
// Gates, decays and the state are in 32-bit: the gates' products take u either in f32 or as three bf16 terms that add up to it.
//
//   decode: one launch.  A workgroup forms u of its whole diagonal block in LDS and takes some of its channels; 16 bytes of weights per lane.
//   blocks: gates (64 tokens x 64 channels a workgroup, on the matrix cores; also the tile's recurrence as ONE factor and ONE input per channel),
//           then the recurrence: every workgroup composes the tiles before its own and walks its 64 tokens, 16 per thread.
// The convolution's history is a ring of `taps` rows: the row that position p takes is none of those it reads.
#include "layered.h"
#include "layered_device.h"

namespace lgh {

constexpr float kGlruRate = -8.0f;
constexpr uint32_t kGlruTile = 64, kGlruLd = kGlruTile + 4, kGlruLdB = kGlruTile + 8;

// decay and input factor of a channel from its two gates' pre-activations
struct GlruStep { float a, x; };
__device__ __forceinline__ GlruStep glru_coef(float rz, float iz, float sp, float u) {
  const float la = kGlruRate * sigmoid_hw(rz) * sp, y = 2.0f * la;
  GlruStep o;
  o.a = exp_hw(la);
  // 1 - exp(y): its series where the difference would cancel (next term below 1e-9 of the value), else from a
  float p = __builtin_fmaf(y, 1.0f / 5040.0f, 1.0f / 720.0f);
  p = __builtin_fmaf(y, p, 1.0f / 120.0f);
  p = __builtin_fmaf(y, p, 1.0f / 24.0f);
  p = __builtin_fmaf(y, p, 1.0f / 6.0f);
  p = __builtin_fmaf(y, p, 0.5f);
  p = __builtin_fmaf(y, p, 1.0f);
  o.x = __builtin_amdgcn_sqrtf(y > -0.25f ? -y * p : __builtin_fmaf(-o.a, o.a, 1.0f)) * sigmoid_hw(iz) * u;
  return o;
}

// ------------------------------------------------------------------------------------------------
// decode; grid (rows of a block / kGlruRows, blocks).  LPR lanes share a row's columns.
// ------------------------------------------------------------------------------------------------
template <uint32_t LPR> constexpr uint32_t glru_rows() { return 4 * (64 / LPR); }   // channels of a workgroup

template <uint32_t LPR>
__global__ void __launch_bounds__(256) glru_step_kernel(const GlruShape s, const GlruBufs b, const int* __restrict__ pos_ptr, float* __restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) float us[];   // [gate_kp]
  const uint32_t tid = threadIdx.x, lane = tid & 63, w = tid >> 6, sub = lane % LPR, blk = blockIdx.y;
  const uint32_t row = blockIdx.x * glru_rows<LPR>() + w * (64 / LPR) + lane / LPR, rc = row < s.bs ? row : s.bs - 1, ch = blk * s.bs + rc;
  const uint32_t c0 = blk * s.bs;
  const int pos = *pos_ptr;
  // weights of this lane's first pass, and what its channel needs at the end, before the convolution
  const uint16_t* wr = b.gates + ((size_t)blk * s.gate_rows + (rc >> 4) * 32 + (rc & 15)) * s.gate_kp;
  const uint16_t* wi = wr + 16 * (size_t)s.gate_kp;
  const uint32_t k0 = sub * 8, kc = k0 < s.gate_kp ? k0 : 0;
  u32x4 pr = ldg_nt128(wr + kc), pi = ldg_nt128(wi + kc);
  const float lam = b.lam[ch], rb = b.rb[ch], ib = b.ib[ch], yv = b.cat[s.off_y + ch], S0 = b.S[ch], xv = b.cat[s.off_x + ch];
  for (uint32_t i = tid; i < s.gate_kp; i += 256) {
    float u = 0.0f;
    if (i < s.bs) {
      const uint32_t c = c0 + i;
      const float* cw = b.conv + (size_t)c * s.taps;
      u = b.conv_b[c];
      for (uint32_t j = s.taps - 1; j >= 1; j--) {   // oldest first
        const bool ok = (int)j <= pos;
        const float h = b.hist[(size_t)(ok ? ((uint32_t)pos - j) % s.taps : 0) * s.width + c];
        u = __builtin_fmaf(ok ? cw[s.taps - 1 - j] : 0.0f, h, u);
      }
      u = __builtin_fmaf(cw[s.taps - 1], b.cat[s.off_x + c], u);
    }
    us[i] = u;
  }
  __syncthreads();
  float r = 0.0f, g = 0.0f;
  for (uint32_t k = k0; k < s.gate_kp; k += LPR * 8) {
    float fr[8], fi[8];
    unpack_row<__bf16, 8>(pr, fr);
    unpack_row<__bf16, 8>(pi, fi);
    const uint32_t kn = k + LPR * 8;
    if (kn < s.gate_kp) { pr = ldg_nt128(wr + kn); pi = ldg_nt128(wi + kn); }
    const f32x4 u0 = *reinterpret_cast<const f32x4*>(us + k), u1 = *reinterpret_cast<const f32x4*>(us + k + 4);
#pragma unroll
    for (int e = 0; e < 4; e++) {
      r = __builtin_fmaf(fr[e], u0[e], r); r = __builtin_fmaf(fr[4 + e], u1[e], r);
      g = __builtin_fmaf(fi[e], u0[e], g); g = __builtin_fmaf(fi[4 + e], u1[e], g);
    }
  }
  r = lanes_sum<LPR>(r);
  g = lanes_sum<LPR>(g);
  if (sub == 0 && row < s.bs) {
    const GlruStep c = glru_coef(r + rb, g + ib, softplus_f(lam), us[row]);
    const float S = __builtin_fmaf(c.a, pos ? S0 : 0.0f, c.x);   // at position 0 whatever is stored belongs to another sequence
    b.S[ch] = S;
    b.hist[(size_t)((uint32_t)pos % s.taps) * s.width + ch] = xv;
    out[ch] = S * gelu_tanh_hw(yv);
  }
}

static bool glru_ok(const GlruShape& s) {
  return s.width && s.blocks && s.bs && (uint64_t)s.blocks * s.bs == s.width && s.taps && s.gate_kp % 64 == 0 && s.gate_kp >= s.bs && s.gate_kp <= kLinMvMaxK &&
         s.gate_rows % 32 == 0 && s.gate_rows >= 2 * s.bs;
}

template <uint32_t LPR>
static hipError_t glru_step_go(const GlruShape& s, const GlruBufs& b, const int* pos_ptr, float* out, hipStream_t st) {
  static bool opted[64] = {};
  if (hipError_t e = lds_opt_in(reinterpret_cast<const void*>(&glru_step_kernel<LPR>), 152 * 1024, opted); e != hipSuccess) return e;
  hipLaunchKernelGGL((glru_step_kernel<LPR>), dim3((s.bs + glru_rows<LPR>() - 1) / glru_rows<LPR>(), s.blocks), dim3(256), (size_t)s.gate_kp * 4, st, s, b, pos_ptr, out);
  return hipGetLastError();
}

hipError_t glru_step_launch(const GlruShape& s, const GlruBufs& b, const int* pos_ptr, float* out, hipStream_t st) {
  if (!glru_ok(s) || !pos_ptr || !out) return hipErrorInvalidValue;
  // lanes per row: one pass over the columns, but workgroups enough for the chip
  if (s.gate_kp <= 64 && s.width >= 64 * kNumCU) return glru_step_go<8>(s, b, pos_ptr, out, st);
  if (s.gate_kp <= 128 && s.width >= 32 * kNumCU) return glru_step_go<16>(s, b, pos_ptr, out, st);
  if (s.gate_kp <= 256) return glru_step_go<32>(s, b, pos_ptr, out, st);
  return glru_step_go<64>(s, b, pos_ptr, out, st);
}

// ------------------------------------------------------------------------------------------------
// blocks: gates.  grid (token tiles, 64-channel tiles of the diagonal blocks); wave w: 16 channels, all 64 tokens
// ------------------------------------------------------------------------------------------------
// the convolution's input of channel c at token t of the block (t may lie before it)
__device__ __forceinline__ float glru_x(const GlruShape& s, const GlruBufs& b, uint32_t pos0, int t, uint32_t c) {
  if (t >= 0) return b.cat[(size_t)t * s.ldcat + s.off_x + c];
  const int p = (int)pos0 + t;
  return p >= 0 ? b.hist[(size_t)((uint32_t)p % s.taps) * s.width + c] : 0.0f;
}

template <class T>
__global__ void __launch_bounds__(256, 3) glru_gates_kernel(const GlruShape s, const GlruBufs b, uint32_t pos0, uint32_t M) {
  constexpr bool BF = sizeof(T) == 2;
  // the columns' u, as the products' operand: f32, or three bf16 terms; later the tile's factors
  __shared__ __attribute__((aligned(16))) uint8_t mem[BF ? 3 * kGlruTile * kGlruLdB * 2 : kGlruTile * kGlruLd * 4];
  __shared__ __attribute__((aligned(16))) float own[kGlruTile][kGlruLd];   // u of the workgroup's own channels; later the tile's inputs, each in place of its u
  __shared__ float part[4][kGlruTile][2];
  const uint32_t tid = threadIdx.x, lane = tid & 63, w = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6)), r16 = lane & 15, g = lane >> 4;
  const uint32_t tiles = (s.bs + 63) / 64, blk = blockIdx.y / tiles, rt = blockIdx.y % tiles, t0 = blockIdx.x * kGlruTile, cb = blk * s.bs;
  const uint32_t rows16 = s.gate_rows / 32, ct = rt * 4 + w, ctc = ct < rows16 ? ct : rows16 - 1;   // this wave's tile of 16 channels
  const uint16_t* wr = b.gates + ((size_t)blk * s.gate_rows + ctc * 32 + r16) * s.gate_kp + g * Frag<T>::PER;
  const uint16_t* wi = wr + 16 * (size_t)s.gate_kp;
  f32x4 ar[4], ai[4];
#pragma unroll
  for (int j = 0; j < 4; j++) { ar[j] = (f32x4)(0.0f); ai[j] = (f32x4)(0.0f); }
  const int tw = (int)(t0 + w * 16);
  // u of 16 tokens of channel 64 kc + lane
  auto load_u = [&](uint32_t kc, float* u) {
    const uint32_t c = kc * 64 + lane, cc = cb + (c < s.bs ? c : s.bs - 1);
    if (s.taps <= 4) {                          // a window of inputs in registers
      float x[19], f[4];
      const float bias = b.conv_b[cc];
#pragma unroll
      for (int i = 0; i < 4; i++) f[i] = (int)s.taps - 1 - i >= 0 ? b.conv[(size_t)cc * s.taps + (s.taps - 1 - i)] : 0.0f;   // f[i]: i positions back
      if (tw > 0) {
        const float* p = b.cat + (size_t)(tw - 3) * s.ldcat + s.off_x + cc;
        if (tw + 16 <= (int)M) {
#pragma unroll
          for (int i = 0; i < 19; i++) x[i] = p[(size_t)i * s.ldcat];
        } else {
#pragma unroll
          for (int i = 0; i < 19; i++) x[i] = b.cat[(size_t)(tw + i - 3 < (int)M ? tw + i - 3 : (int)M - 1) * s.ldcat + s.off_x + cc];
        }
      } else {
#pragma unroll
        for (int i = 0; i < 19; i++) x[i] = i >= 3 || (int)s.taps > 3 - i ? glru_x(s, b, pos0, i - 3 < (int)M ? i - 3 : (int)M - 1, cc) : 0.0f;
      }
#pragma unroll
      for (int i = 0; i < 16; i++) u[i] = __builtin_fmaf(f[0], x[i + 3], __builtin_fmaf(f[1], x[i + 2], __builtin_fmaf(f[2], x[i + 1], __builtin_fmaf(f[3], x[i], bias))));
    } else {
#pragma unroll
      for (int i = 0; i < 16; i++) u[i] = b.conv_b[cc];
      for (uint32_t j = 0; j < s.taps; j++) {
        const float f = b.conv[(size_t)cc * s.taps + (s.taps - 1 - j)];
#pragma unroll
        for (int i = 0; i < 16; i++) {
          const int t = tw + i - (int)j, tc = t < (int)M ? t : (int)M - 1;
          u[i] = __builtin_fmaf(f, glru_x(s, b, pos0, tc, cc), u[i]);
        }
      }
    }
  };
  constexpr int NQ = 64 / Frag<T>::KU;
  struct Wf { u32x4 r[BF ? NQ : 1], i[BF ? NQ : 1]; u32x2 r2[BF ? 1 : NQ], i2[BF ? 1 : NQ]; };   // weights of 64 columns: f32 products take 4 values a unit
  auto load_w = [&](uint32_t kc, Wf& o) {
#pragma unroll
    for (int q = 0; q < NQ; q++) {
      const uint32_t k = kc * 64 + q * Frag<T>::KU;
      if constexpr (BF) { o.r[q] = *reinterpret_cast<const u32x4*>(wr + k); o.i[q] = *reinterpret_cast<const u32x4*>(wi + k); }
      else { o.r2[q] = *reinterpret_cast<const u32x2*>(wr + k); o.i2[q] = *reinterpret_cast<const u32x2*>(wi + k); }
    }
  };
  float u[16];
  Wf wf;
  load_w(0, wf);
  load_u(0, u);
  const uint32_t chunks = s.gate_kp / 64;
  for (uint32_t kc = 0; kc < chunks; kc++) {
    const bool in = kc * 64 + lane < s.bs;
    __syncthreads();                            // the operand before is used up
#pragma unroll
    for (int i = 0; i < 16; i++) {
      const float v = in ? u[i] : 0.0f;
      const uint32_t t = w * 16 + i;
      if (kc == rt) own[t][lane] = v;
      if constexpr (BF) {
        __bf16* o = reinterpret_cast<__bf16*>(mem) + t * kGlruLdB + lane;
        const __bf16 h = (__bf16)v;
        const float v1 = v - (float)h;
        const __bf16 m = (__bf16)v1;
        o[0] = h;
        o[kGlruTile * kGlruLdB] = m;
        o[2 * kGlruTile * kGlruLdB] = (__bf16)(v1 - (float)m);
      } else {
        reinterpret_cast<float*>(mem)[t * kGlruLd + lane] = v;
      }
    }
    __syncthreads();
    const Wf cw = wf;
    if (kc + 1 < chunks) { load_w(kc + 1, wf); load_u(kc + 1, u); }
#pragma unroll
    for (int q = 0; q < NQ; q++) {
      typename Frag<T>::V fr, fi;
      if constexpr (BF) {
        fr = __builtin_bit_cast(bf16x8, cw.r[q]);
        fi = __builtin_bit_cast(bf16x8, cw.i[q]);
      } else {
        fr.x = bf_lo(cw.r2[q].x); fr.y = bf_hi(cw.r2[q].x); fr.z = bf_lo(cw.r2[q].y); fr.w = bf_hi(cw.r2[q].y);
        fi.x = bf_lo(cw.i2[q].x); fi.y = bf_hi(cw.i2[q].x); fi.z = bf_lo(cw.i2[q].y); fi.w = bf_hi(cw.i2[q].y);
      }
#pragma unroll
      for (int j = 0; j < 4; j++) {
        if constexpr (BF) {
#pragma unroll
          for (int p = 2; p >= 0; p--) {        // smallest terms first
            const bf16x8 xf = Frag<T>::load(reinterpret_cast<const __bf16*>(mem) + (p * kGlruTile + j * 16 + r16) * kGlruLdB + q * 32 + g * 8);
            ar[j] = Frag<T>::mma(fr, xf, ar[j]);
            ai[j] = Frag<T>::mma(fi, xf, ai[j]);
          }
        } else {
          const f32x4 xf = *reinterpret_cast<const f32x4*>(reinterpret_cast<const float*>(mem) + (j * 16 + r16) * kGlruLd + q * 16 + g * 4);
          ar[j] = Frag<T>::mma(fr, xf, ar[j]);
          ai[j] = Frag<T>::mma(fi, xf, ai[j]);
        }
      }
    }
  }
  __syncthreads();
  float* fa = reinterpret_cast<float*>(mem);
  float* fx = &own[0][0];
  // lane: channels 4g .. 4g + 3 of the wave's tile, token r16 of token tile j
  const uint32_t cl = w * 16 + g * 4;           // within the 64
  float sp[4], rb[4], ib[4];
#pragma unroll
  for (int e = 0; e < 4; e++) {
    const uint32_t c = rt * 64 + cl + e, cc = cb + (c < s.bs ? c : s.bs - 1);
    sp[e] = softplus_f(b.lam[cc]); rb[e] = b.rb[cc]; ib[e] = b.ib[cc];
  }
#pragma unroll
  for (int j = 0; j < 4; j++) {
    const uint32_t t = j * 16 + r16;
    const f32x4 u = *reinterpret_cast<const f32x4*>(&own[t][cl]);
    f32x4 va, vx;
#pragma unroll
    for (int e = 0; e < 4; e++) {
      const GlruStep c = glru_coef(ar[j][e] + rb[e], ai[j][e] + ib[e], sp[e], u[e]);
      va[e] = t0 + t < M ? c.a : 1.0f;          // behind the block's last token nothing changes
      vx[e] = t0 + t < M ? c.x : 0.0f;
    }
    *reinterpret_cast<f32x4*>(fa + t * kGlruLd + cl) = va;
    *reinterpret_cast<f32x4*>(fx + t * kGlruLd + cl) = vx;
  }
  __syncthreads();
  // thread: channel `lane`, tokens 16 w ..
  const uint32_t c = rt * 64 + lane, cc = cb + c;
  const bool live = c < s.bs;
  float A = 1.0f, X = 0.0f;
#pragma unroll
  for (int i = 0; i < 16; i++) {
    const uint32_t t = w * 16 + i;
    const float a = fa[t * kGlruLd + lane], x = fx[t * kGlruLd + lane];
    A *= a;
    X = __builtin_fmaf(a, X, x);
    if (live && t0 + t < M) {
      b.a[(size_t)(t0 + t) * s.width + cc] = a;
      b.x[(size_t)(t0 + t) * s.width + cc] = x;
    }
  }
  part[w][lane][0] = A;
  part[w][lane][1] = X;
  __syncthreads();
  if (w == 0 && live) {
#pragma unroll
    for (int k = 1; k < 4; k++) {
      A *= part[k][lane][0];
      X = __builtin_fmaf(part[k][lane][0], X, part[k][lane][1]);
    }
    float* o = b.sum + ((size_t)blockIdx.x * s.width + cc) * 2;
    o[0] = A;
    o[1] = X;
    if (blockIdx.x == 0) b.s0[cc] = pos0 ? b.S[cc] : 0.0f;
  }
}

// the recurrence; grid (64-channel tiles, token tiles).  Thread: one channel, 16 tokens
template <class T>
__global__ void __launch_bounds__(256) glru_scan_kernel(const GlruShape s, const GlruBufs b, uint32_t pos0, uint32_t M, T* __restrict__ out, uint32_t ldo) {
  __shared__ float part[4][kGlruTile][2];
  const uint32_t lane = threadIdx.x & 63, w = threadIdx.x >> 6, c = blockIdx.x * 64 + lane, cc = c < s.width ? c : s.width - 1, tile = blockIdx.y, t0 = tile * kGlruTile;
  float a[16], x[16], y[16];
#pragma unroll
  for (int i = 0; i < 16; i++) {
    const uint32_t t = t0 + w * 16 + i, tc = t < M ? t : M - 1;
    a[i] = b.a[(size_t)tc * s.width + cc];
    x[i] = b.x[(size_t)tc * s.width + cc];
    y[i] = b.cat[(size_t)tc * s.ldcat + s.off_y + cc];
    if (t >= M) { a[i] = 1.0f; x[i] = 0.0f; }
  }
  float A = 1.0f, X = 0.0f;
#pragma unroll
  for (int i = 0; i < 16; i++) { A *= a[i]; X = __builtin_fmaf(a[i], X, x[i]); }
  part[w][lane][0] = A;
  part[w][lane][1] = X;
  float S = b.s0[cc];
  for (uint32_t k0 = 0; k0 < tile; k0 += 8) {   // the tiles before, eight in flight
    f32x2 v[8];
#pragma unroll
    for (uint32_t k = 0; k < 8; k++) v[k] = *reinterpret_cast<const f32x2*>(b.sum + ((size_t)(k0 + k < tile ? k0 + k : k0) * s.width + cc) * 2);
#pragma unroll
    for (uint32_t k = 0; k < 8; k++)
      if (k0 + k < tile) S = __builtin_fmaf(v[k].x, S, v[k].y);
  }
  __syncthreads();
  for (uint32_t k = 0; k < w; k++) S = __builtin_fmaf(part[k][lane][0], S, part[k][lane][1]);
  const bool live = c < s.width;
#pragma unroll
  for (int i = 0; i < 16; i++) {
    const uint32_t t = t0 + w * 16 + i;
    S = __builtin_fmaf(a[i], S, x[i]);
    if (live && t < M) out[(size_t)t * ldo + c] = to_act<T>(S * gelu_tanh_hw(y[i]));
  }
  if (tile + 1 == gridDim.y && live) {          // what the sequence keeps
    if (w == 3) b.S[c] = S;
    const uint32_t n = M < s.taps ? M : s.taps;
    for (uint32_t i = w; i < n; i += 4) {
      const uint32_t t = M - 1 - i;
      b.hist[(size_t)((pos0 + t) % s.taps) * s.width + c] = b.cat[(size_t)t * s.ldcat + s.off_x + c];
    }
  }
}

template <class T>
static hipError_t glru_block_go(const GlruShape& s, const GlruBufs& b, uint32_t pos0, uint32_t M, void* out, uint32_t ldo, hipStream_t st) {
  const uint32_t tiles = (M + kGlruTile - 1) / kGlruTile;
  hipLaunchKernelGGL(glru_gates_kernel<T>, dim3(tiles, s.blocks * ((s.bs + 63) / 64)), dim3(256), 0, st, s, b, pos0, M);
  hipLaunchKernelGGL(glru_scan_kernel<T>, dim3((s.width + 63) / 64, tiles), dim3(256), 0, st, s, b, pos0, M, (T*)out, ldo);
  return hipGetLastError();
}

hipError_t glru_block_launch(const GlruShape& s, const GlruBufs& b, uint32_t pos0, uint32_t M, bool f32, void* out, uint32_t ldo, hipStream_t st) {
  if (!glru_ok(s) || M == 0 || ldo < s.width || !b.a || !b.x || !b.sum || !b.s0 || s.blocks * ((s.bs + 63) / 64) > 65535) return hipErrorInvalidValue;
  return f32 ? glru_block_go<float>(s, b, pos0, M, out, ldo, st) : glru_block_go<__bf16>(s, b, pos0, M, out, ldo, st);
}

}  // namespace lgh
