// latent_attention.hip — attention over a shared low-rank latent (layered.h).  A cached position is ONE row for all heads: the normed
// latent c (rank values) and a rotated key part.  Per head k = [W_uk c | rotated part], v = W_uv c.
//
//   decode and short portions ("absorbed"): q . W_uk c = (W_uk^T q) . c, so the key expansion moves to the query and the value
//     expansion behind the weighted sum; (token, head) pairs are the rows of one product against the cached rows, read once for all heads.
//   long portions ("expanded"): keys and values of the context are formed per head by two block products, then ordinary causal attention.
//
// Scores, softmax and the weighted sums are in 32-bit; operands of the matrix cores are the cache's type (bf16 or f32).
#include "layered.h"
#include "layered_device.h"

#include <algorithm>

namespace lgh {

constexpr float kNegHuge = -1e30f, kNegRef = -1e25f, kLog2e = 1.4426950408889634f;

// value i (below rot_n) of a rotated part
__device__ __forceinline__ float rot_value(const LatentShape& s, const float* src, const float* cs, uint32_t i) {
  const uint32_t half = s.rot_n / 2, p = s.halves ? (i < half ? i : i - half) : i >> 1;   // its pair
  const bool second = s.halves ? i >= half : i & 1;
  const float u = src[s.halves ? p : 2 * p], v = src[s.halves ? p + half : 2 * p + 1], c = cs[2 * p], n = cs[2 * p + 1];
  return second ? v * c + u * n : u * c - v * n;
}

// the first key that position i sees; never falls with i
__host__ __device__ __forceinline__ uint32_t lat_key_start(uint32_t window, uint32_t i) { return i >= window ? i - window + 1 : 0; }
uint32_t latent_key_start(const LatentShape& s, uint32_t i) { return lat_key_start(s.window, i); }

// cache row of token t: RMS norm of the latent, rotation of the shared key part.  One workgroup.
template <class T>
__device__ __forceinline__ void latent_cache_row(const LatentShape& s, const LatentBufs& b, const float* dkv, uint32_t pos, float* red) {
  T* row = reinterpret_cast<T*>(b.cache) + (size_t)pos * s.ldc;
  float ss = 0.0f;
  for (uint32_t i = threadIdx.x; i < s.rank; i += 256) ss = __builtin_fmaf(dkv[i], dkv[i], ss);
  const float inv = 1.0f / __builtin_sqrtf(block_sum(ss, red) / (float)s.rank + s.eps);
  for (uint32_t i = threadIdx.x; i < s.rank; i += 256) row[i] = to_act<T>(dkv[i] * inv * b.dkv_norm[i]);
  const float* cs = b.cs + (size_t)pos * s.rot_n;
  for (uint32_t i = threadIdx.x; i < s.rot_dim; i += 256) {
    float v = dkv[s.rank + i];
    if (i < s.rot_n) v = rot_value(s, dkv + s.rank, cs, i);
    row[s.rank + i] = to_act<T>(v);
  }
}

// absorbed queries: grid (chunks of 64 latent rows, heads + 1, tokens); the extra head writes the cache row
template <class T>
__global__ void __launch_bounds__(256) latent_prep_kernel(const LatentShape s, const LatentBufs b, const int* __restrict__ pos_ptr, uint32_t pos0) {
  __shared__ float red[16];
  extern __shared__ float qn[];   // [dimp]
  const uint32_t t = blockIdx.z, h = blockIdx.y, tid = threadIdx.x;
  const uint32_t pos = (pos_ptr ? (uint32_t)*pos_ptr : pos0) + t;
  const float* cat = b.cat + (size_t)t * s.ldcat;
  if (h == s.heads) {
    if (blockIdx.x == 0) latent_cache_row<T>(s, b, cat + s.off_dkv, pos, red);
    return;
  }
  const float* q = b.q + (size_t)t * s.ldq + (size_t)h * (s.dim + s.rot_dim);
  T* qa = reinterpret_cast<T*>(b.qa) + ((size_t)t * s.heads + h) * s.ldc;
  for (uint32_t i = tid; i < s.dimp; i += 256) qn[i] = i < s.dim ? q[i] : 0.0f;
  __syncthreads();
  const uint32_t sub = tid & 15;
  const uint16_t* W = b.uk_t + (size_t)h * s.rank * s.dimp;
#pragma unroll
  for (int it = 0; it < 4; it++) {
    const uint32_t r = blockIdx.x * 64 + it * 16 + (tid >> 4);
    float acc = 0.0f;
    if (r < s.rank) {
      for (uint32_t d = sub * 8; d < s.dimp; d += 128) {
        const u32x4 w = *reinterpret_cast<const u32x4*>(W + (size_t)r * s.dimp + d);
        const float* x = qn + d;
        acc = __builtin_fmaf(bf_lo(w.x), x[0], acc); acc = __builtin_fmaf(bf_hi(w.x), x[1], acc);
        acc = __builtin_fmaf(bf_lo(w.y), x[2], acc); acc = __builtin_fmaf(bf_hi(w.y), x[3], acc);
        acc = __builtin_fmaf(bf_lo(w.z), x[4], acc); acc = __builtin_fmaf(bf_hi(w.z), x[5], acc);
        acc = __builtin_fmaf(bf_lo(w.w), x[6], acc); acc = __builtin_fmaf(bf_hi(w.w), x[7], acc);
      }
    }
    acc += dpp_f<0xB1>(acc); acc += dpp_f<0x4E>(acc); acc += dpp_f<0x141>(acc); acc += dpp_f<0x140>(acc);   // 16 lanes
    if (r < s.rank && sub == 0) qa[r] = to_act<T>(acc);
  }
  if (blockIdx.x == 0) {
    const float* cs = b.cs + (size_t)pos * s.rot_n;
    for (uint32_t i = tid; i < s.ldc - s.rank; i += 256) {
      float v = i < s.rot_dim ? q[s.dim + i] : 0.0f;
      if (i < s.rot_n) v = rot_value(s, q + s.dim, cs, i);
      qa[s.rank + i] = to_act<T>(v);
    }
  }
}

hipError_t latent_prep_launch(const LatentShape& s, const LatentBufs& b, const int* pos_ptr, uint32_t pos0, uint32_t M, bool f32, hipStream_t st) {
  if (s.dimp % 8 || s.ldc < s.rank + s.rot_dim || s.rot_n > s.rot_dim || !b.q || (uint64_t)M * s.heads > kLatAbsorbRows) return hipErrorInvalidValue;
  const dim3 grid((s.rank + 63) / 64, s.heads + 1, M);
  if (f32) hipLaunchKernelGGL(latent_prep_kernel<float>, grid, dim3(256), s.dimp * 4, st, s, b, pos_ptr, pos0);
  else hipLaunchKernelGGL(latent_prep_kernel<__bf16>, grid, dim3(256), s.dimp * 4, st, s, b, pos_ptr, pos0);
  return hipGetLastError();
}

// ------------------------------------------------------------------------------------------------
// absorbed attention.  A workgroup = 16 (token, head) rows x one split of the keys x up to 512 latent columns of the output; 32 keys
// at a time go to LDS by DMA (16-byte chunks of a row stored at chunk ^ (row & 7)).  Everything transposed, as in the expanded kernel
// below: S^T = C Q^T leaves a lane with one row's scores of 8 keys, which is the B operand of O^T = C^T P^T.  Every wave forms all the
// scores (cheaper than exchanging them: one barrier per tile) and owns a quarter of the columns, whose values it takes straight from
// the key tile (the latent IS the value), transposed on the way out of LDS.  With bf16 rows two TEAMS of 4 waves take alternate tiles —
// a tile is a chain of short dependent steps, the other team's fill it — and are merged at the end.
// ------------------------------------------------------------------------------------------------
constexpr uint32_t kLatKeys = 32;

template <class T> constexpr int lat_teams() { return sizeof(T) == 2 ? 2 : 1; }   // (f32 query rows leave no registers for a second wave per SIMD)
template <class T, int NCT> constexpr int lat_units() { return (NCT * 64 + 64) / Frag<T>::KU; }   // units of a query row kept in registers

// NCT: 16-column tiles of the output per wave; nbuf: tile buffers per team; q_alias: the queries pass through the last buffer
template <class T, int NCT>
__global__ void __launch_bounds__(256 * lat_teams<T>()) latent_attn_kernel(const LatentShape s, const LatentBufs b, const int* __restrict__ pos_ptr, uint32_t pos0,
                                                                           uint32_t M, uint32_t n_splits, uint32_t nbuf, uint32_t q_alias) {
  constexpr bool BF = sizeof(T) == 2;
  constexpr uint32_t KT = kLatKeys, PER = Frag<T>::PER;
  constexpr int QU = lat_units<T, NCT>(), TM = lat_teams<T>();  // (a longer query row's rest is read from LDS)
  extern __shared__ __attribute__((aligned(16))) uint8_t smem[];
  const uint32_t lane = threadIdx.x & 63, wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6)), w = wave & 3, team = wave >> 2;
  const uint32_t r16 = lane & 15, g = lane >> 4;
  const uint32_t rows = M * s.heads, row0 = blockIdx.y * 16, sp = blockIdx.x, col0 = blockIdx.z * (NCT * 64);   // (a split's row tiles on one XCD when the splits are a multiple of 8)
  const uint32_t p0 = pos_ptr ? (uint32_t)*pos_ptr : pos0;
  const uint32_t kv = p0 + M, tile0 = lat_key_start(s.window, p0) / KT;   // keys up to kv - 1, from the first token's first visible one on
  const uint32_t tiles = (kv + KT - 1) / KT, per = (tiles - tile0 + n_splits - 1) / n_splits;
  const uint32_t tb = tile0 + sp * per, te = tb + per < tiles ? tb + per : tiles;
  if (tb >= te) return;                                         // (the merge skips the same splits)
  const uint32_t ld = s.ldc, cpr = ld / PER, nu = cpr / 4;      // 16-byte chunks (a multiple of 8) and units of a row
  T* Cs = reinterpret_cast<T*>(smem) + (q_alias ? 0 : 16 * ld); // [team][nbuf][KT][ld]
  T* Qs = q_alias ? Cs + (TM * nbuf - 1) * KT * ld : reinterpret_cast<T*>(smem);   // [16][ld]
  Cs += team * nbuf * KT * ld;
  const T* qg = reinterpret_cast<const T*>(b.qa);
  const T* cg = reinterpret_cast<const T*>(b.cache);
  const uint32_t cs_addr = (uint32_t)__builtin_amdgcn_readfirstlane((int)lds_addr_of(Cs)), qs_addr = (uint32_t)__builtin_amdgcn_readfirstlane((int)lds_addr_of(Qs));
  // this lane's first 16-byte chunk of a tile, and the step to its next one (4 waves x 64 lanes further)
  const uint32_t sr0 = (w * 64 + lane) / cpr, sc0 = (w * 64 + lane) % cpr, dr = 256 / cpr, dc = 256 % cpr;
  auto stage = [&](uint32_t tl, uint32_t buf) {
    const uint32_t dst = cs_addr + buf * KT * ld * (uint32_t)sizeof(T);
    uint32_t r = sr0, ch = sc0;
    for (uint32_t i = w; i < KT * cpr / 64; i += 4) {
      const uint32_t kk = tl * KT + r < kv ? tl * KT + r : kv - 1;
      lds_dma16_untracked(cg + (size_t)kk * ld + (ch ^ (r & 7)) * PER, dst + i * 1024);
      r += dr;
      ch += dc;
      if (ch >= cpr) { ch -= cpr; r++; }
    }
  };
  for (uint32_t i = wave; i < 16 * cpr / 64; i += 4 * TM) {     // the queries, same layout
    const uint32_t c = i * 64 + lane, r = c / cpr, ch = (c % cpr) ^ (r & 7), rr = row0 + r < rows ? row0 + r : rows - 1;
    lds_dma16_untracked(qg + (size_t)rr * ld + ch * PER, qs_addr + i * 1024);
  }
  // nbuf - 1 tiles are under way ahead of the one in use (a wave's share of a tile: cpr / 8 DMA instructions)
  const uint32_t ahead = nbuf > 1 ? nbuf - 1 : 1;
  const uint32_t t_first = tb + team;
  for (uint32_t i = 0; i < ahead && t_first + i * TM < te; i++) stage(t_first + i * TM, i);
  const uint32_t row = row0 + r16 < rows ? row0 + r16 : rows - 1;   // this lane's (token, head) row
  const uint32_t lim = p0 + row / s.heads + 1, low = lat_key_start(s.window, lim - 1);   // keys it sees: low .. lim - 1
  // bf16: scores in units of log2 (one v_exp per weight); f32: natural, with the library exponential
  const float scl = BF ? s.scale * kLog2e : s.scale;
  auto ex = [](float x) { return BF ? __builtin_amdgcn_exp2f(x) : expf(x); };
  float m = kNegHuge, l = 0.0f;
  f32x4 o[NCT];
#pragma unroll
  for (int i = 0; i < NCT; i++) o[i] = (f32x4)(0.0f);
  const uint32_t wc = col0 + w * NCT * 16;
  wait_vm(ahead > 1 && t_first + TM < te ? cpr / 8 : 0);
  __syncthreads();
  auto chunk_at = [&](uint32_t u) { return ((u * 4 + g) ^ (r16 & 7)) * PER; };
  typename Frag<T>::V qr[QU];
#pragma unroll
  for (int u = 0; u < QU; u++) {
    qr[u] = Frag<T>::load(Qs + r16 * ld + chunk_at((uint32_t)u < nu ? u : 0));
    if ((uint32_t)u >= nu) qr[u] = Frag<T>::zero();   // (a shorter row: its first unit again, times 0 — no branches between the loads)
  }
  if (q_alias) __syncthreads();   // the queries' buffer is free
  const uint32_t rounds = (te - tb + TM - 1) / TM;
  uint32_t cur = 0;
  for (uint32_t rd = 0; rd < rounds; rd++, cur = cur + 1 < nbuf ? cur + 1 : 0) {
    const uint32_t tl = t_first + rd * TM, k0 = tl * KT;
    if (nbuf > 1 && tl + ahead * TM < te) stage(tl + ahead * TM, cur + ahead < nbuf ? cur + ahead : cur + ahead - nbuf);
    if (tl < te) {   // (the last round may have a tile for the first team only)
    const T* tile = Cs + cur * KT * ld;
    const T* ka = tile + r16 * ld;
    f32x4 sa[2] = {(f32x4)(0.0f), (f32x4)(0.0f)};
    // two units' key fragments are read while the two before them are multiplied
    typename Frag<T>::V kf[2][4];
    auto read2 = [&](int u, typename Frag<T>::V* k) {
#pragma unroll
      for (int i = 0; i < 2; i++) {
        const uint32_t c = chunk_at((uint32_t)(u + i) < nu ? u + i : 0);
        k[2 * i] = Frag<T>::load(ka + c);
        k[2 * i + 1] = Frag<T>::load(ka + 16 * ld + c);
      }
    };
    static_assert(QU % 2 == 0, "units in pairs");
    read2(0, kf[0]);
#pragma unroll
    for (int u = 0; u < QU; u += 2) {
      if (u + 2 < QU) read2(u + 2, kf[(u / 2 + 1) & 1]);
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int i = 0; i < 2; i++) {
        sa[0] = Frag<T>::mma(kf[(u / 2) & 1][2 * i], qr[u + i], sa[0]);
        sa[1] = Frag<T>::mma(kf[(u / 2) & 1][2 * i + 1], qr[u + i], sa[1]);
      }
    }
    for (uint32_t u = QU; u < nu; u++) {
      const uint32_t c = chunk_at(u);
      const typename Frag<T>::V q = Frag<T>::load(Qs + r16 * ld + c);
      sa[0] = Frag<T>::mma(Frag<T>::load(ka + c), q, sa[0]);
      sa[1] = Frag<T>::mma(Frag<T>::load(ka + 16 * ld + c), q, sa[1]);
    }
    float m1 = m;
#pragma unroll
    for (int n = 0; n < 2; n++)
#pragma unroll
      for (int e = 0; e < 4; e++) {
        const float v = k0 + n * 16 + g * 4 + e - low < lim - low ? sa[n][e] * scl : kNegHuge;
        sa[n][e] = v;
        m1 = fmaxf(m1, v);
      }
    m1 = fmaxf(m1, __shfl_xor(m1, 16, 64));
    m1 = fmaxf(m1, __shfl_xor(m1, 32, 64));
    const float alpha = ex(m - m1);
    float sum = 0.0f;
#pragma unroll
    for (int n = 0; n < 2; n++)
#pragma unroll
      for (int e = 0; e < 4; e++) {
        const float p = k0 + n * 16 + g * 4 + e - low < lim - low ? ex(sa[n][e] - m1) : 0.0f;
        sa[n][e] = p;
        sum += p;
      }
    l = __builtin_fmaf(l, alpha, sum);   // this lane's keys only; added up at the end
    if (__any(m1 > m)) {
#pragma unroll
      for (int i = 0; i < NCT; i++) o[i] *= alpha;
    }
    m = m1;
    if constexpr (BF) {
      bf16x8 pf;
#pragma unroll
      for (int e = 0; e < 4; e++) { pf[e] = (__bf16)sa[0][e]; pf[4 + e] = (__bf16)sa[1][e]; }
#pragma unroll
      for (int i = 0; i < NCT; i++) {
        const uint32_t c0 = wc + i * 16 < ld ? wc + i * 16 : ld - 16;   // (columns past the row: computed, never stored)
        o[i] = Frag<T>::mma(tile_value_frag<T>(tile, ld, 0, c0, r16, g), pf, o[i]);
      }
    } else {
#pragma unroll
      for (int n = 0; n < 2; n++)
#pragma unroll
        for (int i = 0; i < NCT; i++) {
          const uint32_t c0 = wc + i * 16 < ld ? wc + i * 16 : ld - 16;
          o[i] = Frag<T>::mma(tile_value_frag<T>(tile, ld, n, c0, r16, g), sa[n], o[i]);
        }
    }
    }
    if (nbuf == 1) {
      __syncthreads();
      if (tl + TM < te) stage(tl + TM, 0);
    }
    wait_vm(tl + 2 * TM < te && nbuf > 2 ? cpr / 8 : 0);   // the next tile has arrived; the one after it may be under way
    __syncthreads();
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if constexpr (TM == 2) {   // the second team's share, lane by lane
    f32x4* mo = reinterpret_cast<f32x4*>(smem);                  // [wave][NCT][lane]
    float* mm = reinterpret_cast<float*>(mo + 4 * NCT * 64);     // [wave][2][lane]
    if (team == 1) {
#pragma unroll
      for (int i = 0; i < NCT; i++) mo[(w * NCT + i) * 64 + lane] = o[i];
      mm[w * 128 + lane] = m;
      mm[w * 128 + 64 + lane] = l;
    }
    __syncthreads();
    if (team == 1) return;
    const float om = mm[w * 128 + lane], ol = mm[w * 128 + 64 + lane], mn = fmaxf(m, om), a0 = ex(m - mn), a1 = ex(om - mn);
    l = l * a0 + ol * a1;
    m = mn;
#pragma unroll
    for (int i = 0; i < NCT; i++) {
      const f32x4 x = mo[(w * NCT + i) * 64 + lane];
#pragma unroll
      for (int e = 0; e < 4; e++) o[i][e] = o[i][e] * a0 + x[e] * a1;
    }
  }
  if (row0 + r16 >= rows) return;
  const size_t pr = (size_t)sp * rows + row0 + r16;
  if (w == 0 && g == 0 && blockIdx.z == 0) { b.part_ml[pr * 2] = BF ? m * (1.0f / kLog2e) : m; b.part_ml[pr * 2 + 1] = l; }
#pragma unroll
  for (int i = 0; i < NCT; i++) {
    const uint32_t c = wc + i * 16 + g * 4;
    float* dst = b.part_acc + pr * s.rank + c;
    if (c + 4 <= s.rank && (s.rank & 3) == 0) *reinterpret_cast<f32x4*>(dst) = o[i];
    else
      for (uint32_t e = 0; e < 4; e++)
        if (c + e < s.rank) dst[e] = o[i][e];
  }
}

// how a shape's tiles lie in LDS (bytes 0: a row is too long)
struct LatentPlan { uint32_t nbuf, q_alias; size_t bytes; };
static LatentPlan latent_plan(const LatentShape& s, bool f32) {
  const uint32_t el = f32 ? 4 : 2, teams = f32 ? lat_teams<float>() : lat_teams<__bf16>();
  const size_t row = (size_t)s.ldc * el, tile = kLatKeys * row, merge = 34 * 1024 + 1024;
  const uint32_t nct = (s.rank + 63) / 64, c = nct <= 1 ? 1 : nct <= 2 ? 2 : nct <= 4 ? 4 : 8;   // the kernel's column tiles per wave
  const bool in_regs = s.ldc <= c * 64 + 64;                                                 // the whole query row stays in registers
  for (uint32_t n : {3u, 2u, 1u}) {
    if (16 * row + teams * n * tile <= 155 * 1024) return {n, 0u, std::max(16 * row + teams * n * tile, merge)};
    if (n > 1 && in_regs && teams * n * tile <= 155 * 1024) return {n, 1u, std::max(teams * n * tile, merge)};
  }
  return {0, 0, 0};
}
bool latent_fits(const LatentShape& s, bool f32) { return latent_plan(s, f32).bytes != 0; }

template <class T, int NCT>
static hipError_t latent_attn_go(const LatentShape& s, const LatentBufs& b, const int* pos_ptr, uint32_t pos0, uint32_t M, uint32_t n_splits, const LatentPlan& pl,
                                 uint32_t zs, hipStream_t st) {
  static bool opted[64] = {};
  if (hipError_t e = lds_opt_in(reinterpret_cast<const void*>(&latent_attn_kernel<T, NCT>), 156 * 1024, opted); e != hipSuccess) return e;
  hipLaunchKernelGGL((latent_attn_kernel<T, NCT>), dim3(n_splits, (M * s.heads + 15) / 16, zs), dim3(256 * lat_teams<T>()), pl.bytes, st, s, b, pos_ptr,
                     pos0, M, n_splits, pl.nbuf, pl.q_alias);
  return hipGetLastError();
}

hipError_t latent_attn_launch(const LatentShape& s, const LatentBufs& b, const int* pos_ptr, uint32_t pos0, uint32_t M, uint32_t n_splits, bool f32,
                              hipStream_t st) {
  const LatentPlan pl = latent_plan(s, f32);
  if (!pl.bytes || s.window == 0 || s.ldc % 64 || n_splits == 0 || n_splits > kLatMaxSplits || M == 0 || (uint64_t)M * s.heads > kLatAbsorbRows) return hipErrorInvalidValue;
  const uint32_t nct = (s.rank + 63) / 64;
#define LGH_LAT_CASE(N) return f32 ? latent_attn_go<float, N>(s, b, pos_ptr, pos0, M, n_splits, pl, zs, st) : latent_attn_go<__bf16, N>(s, b, pos_ptr, pos0, M, n_splits, pl, zs, st)
  uint32_t zs = 1;
  if (nct <= 1) LGH_LAT_CASE(1);
  if (nct <= 2) LGH_LAT_CASE(2);
  if (nct <= 4) LGH_LAT_CASE(4);
  zs = (nct + 7) / 8;
  LGH_LAT_CASE(8);
#undef LGH_LAT_CASE
}

// ------------------------------------------------------------------------------------------------
// merge + value expansion + head gate: grid (chunks of 32 value rows, token * heads).  The value rows and the first partial sums are
// requested before the merge weights are known: the kernel is a handful of memory round trips long.
// ------------------------------------------------------------------------------------------------
constexpr int kOutB = 16;   // partial sums in flight per thread

template <class O>
__global__ void __launch_bounds__(512) latent_out_kernel(const LatentShape s, const LatentBufs b, const int* __restrict__ pos_ptr, uint32_t pos0, uint32_t M,
                                                         uint32_t n_splits, O* __restrict__ out, uint32_t ldo) {
  extern __shared__ __attribute__((aligned(16))) float lat[];   // [rankp], with room for the merge's thread groups
  __shared__ float wgt[kLatMaxSplits];
  const uint32_t tid = threadIdx.x, r = blockIdx.y, t = r / s.heads, h = r % s.heads, rows = M * s.heads;
  const uint32_t p0 = pos_ptr ? (uint32_t)*pos_ptr : pos0, kv = p0 + M;
  const uint32_t tiles = (kv + kLatKeys - 1) / kLatKeys - lat_key_start(s.window, p0) / kLatKeys, per = (tiles + n_splits - 1) / n_splits, act = (tiles + per - 1) / per;
  const uint32_t lane = tid & 63, w = tid >> 6;
  static_assert(kLatMaxSplits == 128, "two splits per lane");
  float mi[2], li[2];
#pragma unroll
  for (uint32_t k = 0; k < 2; k++) {
    const uint32_t sp = lane + k * 64, spc = sp < act ? sp : act - 1;
    mi[k] = b.part_ml[((size_t)spc * rows + r) * 2];
    li[k] = b.part_ml[((size_t)spc * rows + r) * 2 + 1] * (sp < act ? 1.0f : 0.0f);   // (an inactive split repeats the last one with weight 0)
  }
  u32x4 wv0[4];   // the wave's 4 value rows, first 512 columns
#pragma unroll
  for (int it = 0; it < 4; it++) {
    const uint32_t v = blockIdx.x * 32 + it * 8 + w, vc = v < s.vdim ? v : s.vdim - 1, k = lane * 8 < s.rankp ? lane * 8 : 0;
    wv0[it] = *reinterpret_cast<const u32x4*>(b.uv + ((size_t)h * s.vdim + vc) * s.rankp + k);
  }
  // 4 columns per thread, the splits dealt to as many thread groups as there are threads for
  const uint32_t quads = s.rankp / 4, groups = quads < 512 ? 512 / quads : 1, grp = tid / quads < groups ? tid / quads : 0;
  const bool vec = (s.rank & 3) == 0;
  auto fetch = [&](uint32_t sp, uint32_t q) -> f32x4 {   // clamped: the loads are unconditional
    const float* src = b.part_acc + ((size_t)(sp < act ? sp : act - 1) * rows + r) * s.rank;
    if (vec) return *reinterpret_cast<const f32x4*>(src + (q * 4 < s.rank ? q * 4 : 0));
    f32x4 v;
#pragma unroll
    for (uint32_t e = 0; e < 4; e++) v[e] = src[q * 4 + e < s.rank ? q * 4 + e : 0];
    return v;
  };
  f32x4 first[kOutB];
  const uint32_t q0 = quads < 512 ? tid % quads : tid;
#pragma unroll
  for (int i = 0; i < kOutB; i++) first[i] = fetch(grp + i * groups, q0 < quads ? q0 : 0);
  {
    const float mm = wave_max(fmaxf(mi[0], mi[1])), f0 = expf(mi[0] - mm), f1 = expf(mi[1] - mm), tot = wave_sum(f0 * li[0] + f1 * li[1]);
    if (w == 0) { wgt[lane] = f0 / tot; wgt[lane + 64] = f1 / tot; }
  }
  __syncthreads();
  f32x4* acc4 = reinterpret_cast<f32x4*>(lat);   // [groups][quads]
  for (uint32_t q = q0; q < quads && tid / quads < groups; q += 512) {
    f32x4 v = (f32x4)(0.0f);
    for (uint32_t sp = grp; sp < act; sp += groups * kOutB) {
#pragma unroll
      for (int i = 0; i < kOutB; i++) {
        const uint32_t k = sp + i * groups;
        const f32x4 x = q == q0 && sp == grp ? first[i] : fetch(k, q);
        const float wg = k < act ? wgt[k] : 0.0f;
#pragma unroll
        for (int e = 0; e < 4; e++) v[e] = __builtin_fmaf(wg, x[e], v[e]);
      }
    }
#pragma unroll
    for (uint32_t e = 0; e < 4; e++)
      if (q * 4 + e >= s.rank) v[e] = 0.0f;
    acc4[grp * quads + q] = v;
  }
  __syncthreads();
  if (groups > 1) {
    f32x4 v = (f32x4)(0.0f);
    if (tid < quads)
      for (uint32_t k = 0; k < groups; k++) v += acc4[k * quads + tid];
    __syncthreads();
    if (tid < quads) acc4[tid] = v;
    __syncthreads();
  }
  const float* gates = b.cat + (size_t)t * s.ldcat + s.off_g;
  float gate[4];
#pragma unroll
  for (int it = 0; it < 4; it++) {
    const uint32_t v = blockIdx.x * 32 + it * 8 + w;
    gate[it] = gates[s.gate_values ? h * s.vdim + (v < s.vdim ? v : 0) : h];
  }
#pragma unroll
  for (int it = 0; it < 4; it++) {
    const uint32_t v = blockIdx.x * 32 + it * 8 + w;
    if (v >= s.vdim) continue;
    const uint16_t* W = b.uv + ((size_t)h * s.vdim + v) * s.rankp;
    float acc = 0.0f;
    for (uint32_t k = lane * 8; k < s.rankp; k += 512) {
      const u32x4 wv = k < 512 ? wv0[it] : *reinterpret_cast<const u32x4*>(W + k);
      const f32x4 x0 = *reinterpret_cast<const f32x4*>(lat + k), x1 = *reinterpret_cast<const f32x4*>(lat + k + 4);
      acc = __builtin_fmaf(bf_lo(wv.x), x0.x, acc); acc = __builtin_fmaf(bf_hi(wv.x), x0.y, acc);
      acc = __builtin_fmaf(bf_lo(wv.y), x0.z, acc); acc = __builtin_fmaf(bf_hi(wv.y), x0.w, acc);
      acc = __builtin_fmaf(bf_lo(wv.z), x1.x, acc); acc = __builtin_fmaf(bf_hi(wv.z), x1.y, acc);
      acc = __builtin_fmaf(bf_lo(wv.w), x1.z, acc); acc = __builtin_fmaf(bf_hi(wv.w), x1.w, acc);
    }
    acc = wave_sum_to_lane63(acc);
    if (lane == 63) out[(size_t)t * ldo + h * s.vdim + v] = to_act<O>(acc * sigmoid_f(gate[it]));
  }
}

hipError_t latent_out_launch(const LatentShape& s, const LatentBufs& b, const int* pos_ptr, uint32_t pos0, uint32_t M, uint32_t n_splits, void* out, uint32_t ldo, bool out_f32, hipStream_t st) {
  if (s.rankp % 8 || n_splits == 0 || n_splits > kLatMaxSplits) return hipErrorInvalidValue;
  const dim3 grid((s.vdim + 31) / 32, M * s.heads), th(512);
  const size_t lds = (size_t)(s.rankp < 2048 ? 2048 : s.rankp) * 4;
  if (out_f32) hipLaunchKernelGGL(latent_out_kernel<float>, grid, th, lds, st, s, b, pos_ptr, pos0, M, n_splits, (float*)out, ldo);
  else hipLaunchKernelGGL(latent_out_kernel<__bf16>, grid, th, lds, st, s, b, pos_ptr, pos0, M, n_splits, (__bf16*)out, ldo);
  return hipGetLastError();
}

// ------------------------------------------------------------------------------------------------
// expanded path: queries, keys and values per head
// ------------------------------------------------------------------------------------------------
bool latent_flash_shape(const LatentShape& s, uint32_t* dq, uint32_t* dvp) {
  const uint32_t d = s.dim + s.rot_dim;
  if (d > 256 || s.vdim > 256) return false;
  *dq = d <= 64 ? 64 : d <= 128 ? 128 : d <= 192 ? 192 : 256;
  *dvp = s.vdim <= 64 ? 64 : s.vdim <= 128 ? 128 : 256;
  return true;
}

// the block's cache rows and queries [head][token][dq] = [unrotated | rotated | zeros]; grid (tokens)
template <class T>
__global__ void __launch_bounds__(256) latent_flash_prep_kernel(const LatentShape s, const LatentBufs b, T* __restrict__ q, uint32_t dq, uint32_t Mcap,
                                                                uint32_t pos0) {
  __shared__ float red[16];
  const uint32_t t = blockIdx.x, pos = pos0 + t;
  const float* cat = b.cat + (size_t)t * s.ldcat;
  latent_cache_row<T>(s, b, cat + s.off_dkv, pos, red);
  const float* cs = b.cs + (size_t)pos * s.rot_n;
  const uint32_t hd = s.dim + s.rot_dim;
  for (uint32_t i = threadIdx.x; i < s.heads * dq; i += 256) {
    const uint32_t h = i / dq, j = i % dq;
    const float* src = b.q + (size_t)t * s.ldq + (size_t)h * hd;
    float v = j < hd ? src[j] : 0.0f;
    if (j >= s.dim && j - s.dim < s.rot_n) v = rot_value(s, src + s.dim, cs, j - s.dim);
    q[((size_t)h * Mcap + t) * dq + j] = to_act<T>(v);
  }
}

// the shared rotated key part of every cached position (cache: from the first one on), beside each head's own key; grid (positions)
template <class T>
__global__ void __launch_bounds__(256) latent_rot_spread_kernel(const LatentShape s, const T* __restrict__ cache, T* __restrict__ k, uint32_t dq, uint64_t Tcap) {
  const uint32_t t = blockIdx.x;
  for (uint32_t i = threadIdx.x; i < s.heads * s.rot_dim; i += 256) {
    const uint32_t h = i / s.rot_dim, j = i % s.rot_dim;
    k[((size_t)h * Tcap + t) * dq + s.dim + j] = cache[(size_t)t * s.ldc + s.rank + j];
  }
}

hipError_t latent_flash_prep_launch(const LatentShape& s, const LatentBufs& b, const LatentFlash& f, uint32_t pos0, uint32_t M, bool f32, hipStream_t st) {
  if (M == 0 || M > f.Mcap || f.base % 64 || f.base > pos0 || pos0 - f.base + M > f.Tcap || f.base > lat_key_start(s.window, pos0) || !b.q) return hipErrorInvalidValue;
  const uint32_t n = pos0 - f.base + M;
  if (f32) {
    hipLaunchKernelGGL(latent_flash_prep_kernel<float>, dim3(M), dim3(256), 0, st, s, b, (float*)f.q, f.dq, f.Mcap, pos0);
    if (s.rot_dim) hipLaunchKernelGGL(latent_rot_spread_kernel<float>, dim3(n), dim3(256), 0, st, s, (const float*)b.cache + (size_t)f.base * s.ldc, (float*)f.k, f.dq, f.Tcap);
  } else {
    hipLaunchKernelGGL(latent_flash_prep_kernel<__bf16>, dim3(M), dim3(256), 0, st, s, b, (__bf16*)f.q, f.dq, f.Mcap, pos0);
    if (s.rot_dim) hipLaunchKernelGGL(latent_rot_spread_kernel<__bf16>, dim3(n), dim3(256), 0, st, s, (const __bf16*)b.cache + (size_t)f.base * s.ldc, (__bf16*)f.k, f.dq, f.Tcap);
  }
  return hipGetLastError();
}

// Causal attention, everything transposed: S^T = K Q^T leaves a lane with one query's scores of keys 4g .. 4g + 3, which is the B
// operand of O^T = V^T P^T when the value fragment's k slots are assigned the same way — the weights never leave the registers.
// A workgroup = 4 waves = 64 * QT queries of one head; K and V^T tiles of KT keys go to LDS by DMA, two buffers.
// two workgroups per CU where their tiles fit LDS
template <class T, int DQ, int DV> constexpr size_t flash_lds() { return 2 * ((sizeof(T) == 2 ? 64 : 32) * (size_t)DQ * sizeof(T) + (size_t)DV * 128); }
template <class T, int DQ, int DV> constexpr int flash_wgs() { return 2 * flash_lds<T, DQ, DV>() <= 160 * 1024 && DV <= 128 ? 2 : 1; }

template <class T, int DQ, int DV>
__global__ void __launch_bounds__(256, (flash_wgs<T, DQ, DV>())) latent_flash_kernel(const LatentShape s, const LatentBufs b, const LatentFlash f, uint32_t pos0, uint32_t M, uint32_t nqb,
                                                           T* __restrict__ out, uint32_t ldo) {
  constexpr bool BF = sizeof(T) == 2;
  constexpr int KT = BF ? 64 : 32, QT = BF ? 2 : 1, NK = KT / 16, NU = DQ / Frag<T>::KU, ND = DV / 16, NP = KT / Frag<T>::KU;
  constexpr uint32_t XC = DQ * sizeof(T) / 16, kK = KT * XC * 16, kV = DV * 128, kBuf = kK + kV;
  extern __shared__ __attribute__((aligned(16))) uint8_t smem[];
  const uint32_t lane = threadIdx.x & 63, w = (uint32_t)__builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6)), r16 = lane & 15, g = lane >> 4;
  // the longest rows first, and of the second half of the grid the shortest first: workgroups i and i + half, which share a CU when the
  // whole grid is resident, then have equal work together
  const uint32_t h = blockIdx.x % s.heads, qi = blockIdx.x / s.heads, hi = (nqb + 1) / 2, qb = qi < hi ? nqb - 1 - qi : qi - hi;
  const uint32_t q0 = qb * 64 * QT, qw = q0 + w * 16 * QT;
  const uint32_t qlast = q0 + 64 * QT - 1 < M - 1 ? q0 + 64 * QT - 1 : M - 1;
  const uint32_t tw = lat_key_start(s.window, pos0 + q0) / KT, tiles = (pos0 + qlast + KT) / KT;   // keys up to pos0 + qlast (positions count from f.base)
  const T* K = reinterpret_cast<const T*>(f.k) + (size_t)h * f.Tcap * DQ;
  const T* V = reinterpret_cast<const T*>(f.vt) + (size_t)h * f.dvp * f.Tcap;
  auto stage = [&](uint32_t tl, uint32_t buf) {
    uint8_t* base = smem + buf * kBuf;
#pragma unroll
    for (int i = 0; i < (int)(kK / 4096); i++) {
      const uint32_t c = (i * 4 + w) * 64 + lane, row = c / XC, ch = (c % XC) ^ (row & 7);
      lds_dma16(K + ((size_t)tl * KT + row) * DQ + ch * (16 / sizeof(T)), base + (i * 4 + w) * 1024);
    }
#pragma unroll
    for (int i = 0; i < (int)(kV / 4096); i++) {
      const uint32_t c = (i * 4 + w) * 64 + lane, row = c / 8, ch = (c % 8) ^ (row & 7);
      lds_dma16(V + (size_t)row * f.Tcap + (size_t)tl * KT + ch * (16 / sizeof(T)), base + kK + (i * 4 + w) * 1024);
    }
  };
  stage(tw, 0);
  typename Frag<T>::V qf[QT][NU];
#pragma unroll
  for (int t = 0; t < QT; t++) {
    const uint32_t m = qw + t * 16 + r16;
    const T* qr = reinterpret_cast<const T*>(f.q) + ((size_t)h * f.Mcap + (m < M ? m : M - 1)) * DQ + g * Frag<T>::PER;
#pragma unroll
    for (int u = 0; u < NU; u++) qf[t][u] = Frag<T>::load(qr + u * Frag<T>::KU);
  }
  f32x4 o[ND][QT];
  float mx[QT], l[QT];
#pragma unroll
  for (int t = 0; t < QT; t++) {
    mx[t] = kNegRef; l[t] = 0.0f;   // (far above a masked score: a query that has seen nothing yet weighs masked keys with 0)
#pragma unroll
    for (int i = 0; i < ND; i++) o[i][t] = (f32x4)(0.0f);
  }
  // bf16: scores in units of log2 (one v_exp per weight); f32: natural, with the library exponential
  const float sc = BF ? s.scale * kLog2e : s.scale;
  __builtin_amdgcn_s_waitcnt(0x0F70);   // vmcnt(0)
  __syncthreads();
  const uint32_t low1 = lat_key_start(s.window, pos0 + qw + 16 * QT - 1);   // (wave-uniform) every query of this wave sees all keys from here to pos0 + qw
  for (uint32_t tl = tw; tl < tiles; tl++) {
    const uint32_t cur = (tl - tw) & 1, k0 = tl * KT;
    if (tl + 1 < tiles) stage(tl + 1, cur ^ 1);
    const uint8_t* kb = smem + cur * kBuf;
    const uint8_t* vb = kb + kK;
    f32x4 sa[NK][QT];
#pragma unroll
    for (int n = 0; n < NK; n++)
#pragma unroll
      for (int t = 0; t < QT; t++) sa[n][t] = (f32x4)(0.0f);
#pragma unroll
    for (int u = 0; u < NU; u++)
#pragma unroll
      for (int n = 0; n < NK; n++) {
        const uint32_t row = n * 16 + r16;
        const typename Frag<T>::V kf = Frag<T>::load(reinterpret_cast<const T*>(kb + row * (XC * 16) + (((uint32_t)(u * 4) + g) ^ (row & 7)) * 16));
#pragma unroll
        for (int t = 0; t < QT; t++) sa[n][t] = Frag<T>::mma(kf, qf[t][u], sa[n][t]);
      }
    if (k0 + KT > pos0 + qw + 1 || k0 < low1) {   // wave-uniform: some key may lie behind some query, or before its window
      asm volatile("");              // (kept a branch: most tiles have no masks to apply)
#pragma unroll
      for (int t = 0; t < QT; t++) {
        const uint32_t lim = pos0 + qw + t * 16 + r16, low = lat_key_start(s.window, lim);   // first and last visible key
#pragma unroll
        for (int n = 0; n < NK; n++)
#pragma unroll
          for (int e = 0; e < 4; e++) sa[n][t][e] = k0 + n * 16 + g * 4 + e - low > lim - low ? kNegHuge : sa[n][t][e];
      }
    }
#pragma unroll
    for (int t = 0; t < QT; t++) {   // maxima of the raw scores; the scale goes into the exponent's multiply-add
      float m1 = mx[t];
#pragma unroll
      for (int n = 0; n < NK; n++)
#pragma unroll
        for (int e = 0; e < 4; e++) m1 = fmaxf(m1, sa[n][t][e]);
      m1 = fmaxf(m1, __shfl_xor(m1, 16, 64));
      m1 = fmaxf(m1, __shfl_xor(m1, 32, 64));
      const float off = -m1 * sc;
      auto weight = [&](float v) { const float x = __builtin_fmaf(v, sc, off); return BF ? __builtin_amdgcn_exp2f(x) : expf((v - m1) * sc); };
      const float a = BF ? __builtin_amdgcn_exp2f((mx[t] - m1) * sc) : expf((mx[t] - m1) * sc);
      float sum = 0.0f;
#pragma unroll
      for (int n = 0; n < NK; n++)
#pragma unroll
        for (int e = 0; e < 4; e++) {
          const float p = weight(sa[n][t][e]);
          sa[n][t][e] = p;
          sum += p;
        }
      l[t] = __builtin_fmaf(l[t], a, sum);
      if (__any(m1 > mx[t])) {
#pragma unroll
        for (int i = 0; i < ND; i++) o[i][t] *= a;
      }
      mx[t] = m1;
    }
#pragma unroll
    for (int u = 0; u < NP; u++) {
      typename Frag<T>::V pf[QT];
#pragma unroll
      for (int t = 0; t < QT; t++) {
        if constexpr (BF) {
#pragma unroll
          for (int e = 0; e < 4; e++) { pf[t][e] = (__bf16)sa[2 * u][t][e]; pf[t][4 + e] = (__bf16)sa[2 * u + 1][t][e]; }
        } else {
          pf[t] = sa[u][t];
        }
      }
#pragma unroll
      for (int i = 0; i < ND; i++) {
        const uint32_t row = i * 16 + r16;
        typename Frag<T>::V vf;
        if constexpr (BF) {
          const bf16x4 a = *reinterpret_cast<const bf16x4*>(vb + row * 128 + (((uint32_t)(4 * u) + (g >> 1)) ^ (row & 7)) * 16 + (g & 1) * 8);
          const bf16x4 c = *reinterpret_cast<const bf16x4*>(vb + row * 128 + (((uint32_t)(4 * u + 2) + (g >> 1)) ^ (row & 7)) * 16 + (g & 1) * 8);
          vf = __builtin_shufflevector(a, c, 0, 1, 2, 3, 4, 5, 6, 7);
        } else {
          vf = Frag<T>::load(reinterpret_cast<const T*>(vb + row * 128 + (((uint32_t)(4 * u) + g) ^ (row & 7)) * 16));
        }
#pragma unroll
        for (int t = 0; t < QT; t++) o[i][t] = Frag<T>::mma(vf, pf[t], o[i][t]);
      }
    }
    __builtin_amdgcn_s_waitcnt(0x0F70);
    __syncthreads();
  }
#pragma unroll
  for (int t = 0; t < QT; t++) {
    float lt = l[t];
    lt += __shfl_xor(lt, 16, 64);
    lt += __shfl_xor(lt, 32, 64);
    const uint32_t m = qw + t * 16 + r16;
    if (m >= M) continue;
    const float* gates = b.cat + (size_t)m * s.ldcat + s.off_g;
    const float fac = (s.gate_values ? 1.0f : sigmoid_f(gates[h])) / lt;
    T* dst = out + (size_t)m * ldo + h * s.vdim;
#pragma unroll
    for (int i = 0; i < ND; i++)
#pragma unroll
      for (int e = 0; e < 4; e++) {
        const uint32_t v = i * 16 + g * 4 + e;
        if (v < s.vdim) dst[v] = to_act<T>(o[i][t][e] * fac * (s.gate_values ? sigmoid_f(gates[h * s.vdim + v]) : 1.0f));
      }
  }
}

template <class T, int DQ, int DV>
static hipError_t latent_flash_go(const LatentShape& s, const LatentBufs& b, const LatentFlash& f, uint32_t pos0, uint32_t M, void* out, uint32_t ldo, hipStream_t st) {
  static bool opted[64] = {};
  constexpr size_t lds = flash_lds<T, DQ, DV>();
  static_assert(lds <= 160 * 1024, "two tiles fit LDS");
  if (hipError_t e = lds_opt_in(reinterpret_cast<const void*>(&latent_flash_kernel<T, DQ, DV>), (int)lds, opted); e != hipSuccess) return e;
  const uint32_t QB = sizeof(T) == 2 ? 128 : 64, nqb = (M + QB - 1) / QB;
  hipLaunchKernelGGL((latent_flash_kernel<T, DQ, DV>), dim3(nqb * s.heads), dim3(256), lds, st, s, b, f, pos0, M, nqb, (T*)out, ldo);
  return hipGetLastError();
}

template <class T>
static hipError_t latent_flash_pick(const LatentShape& s, const LatentBufs& b, const LatentFlash& f, uint32_t pos0, uint32_t M, void* out, uint32_t ldo, hipStream_t st) {
#define LGH_FLASH_CASE(Q, V) if (f.dq == Q && f.dvp == V) return latent_flash_go<T, Q, V>(s, b, f, pos0, M, out, ldo, st);
  LGH_FLASH_CASE(64, 64) LGH_FLASH_CASE(64, 128) LGH_FLASH_CASE(64, 256)
  LGH_FLASH_CASE(128, 64) LGH_FLASH_CASE(128, 128) LGH_FLASH_CASE(128, 256)
  LGH_FLASH_CASE(192, 64) LGH_FLASH_CASE(192, 128) LGH_FLASH_CASE(192, 256)
  LGH_FLASH_CASE(256, 64) LGH_FLASH_CASE(256, 128) LGH_FLASH_CASE(256, 256)
#undef LGH_FLASH_CASE
  return hipErrorInvalidValue;
}

hipError_t latent_flash_launch(const LatentShape& s, const LatentBufs& b, const LatentFlash& f, uint32_t pos0, uint32_t M, bool f32, void* out, uint32_t ldo,
                               hipStream_t st) {
  const uint64_t KT = f32 ? 32 : 64;
  if (M == 0 || M > f.Mcap || f.Tcap % 64 || f.base > pos0 || s.window == 0) return hipErrorInvalidValue;
  pos0 -= f.base;
  if ((pos0 + M + KT - 1) / KT * KT > f.Tcap) return hipErrorInvalidValue;   // whole key tiles are read
  return f32 ? latent_flash_pick<float>(s, b, f, pos0, M, out, ldo, st) : latent_flash_pick<__bf16>(s, b, f, pos0, M, out, ldo, st);
}

}  // namespace lgh
