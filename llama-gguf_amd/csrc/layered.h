// layered.h — models whose layers are described one by one (lgh_layer_desc: a mixer and an optional feed-forward), on the engine's own
// context, step function and graphs (internal).  Kernels: linear_bf16.hip (matrix products), latent_attention.hip, tied_attention.hip,
// gated_attention.hip, mlstm.hip, gla.hip, glru.hip, delta.hip, moe_route.hip (routing of the experts), layered_misc.hip (embedding, norms, residual updates); layered.hip assembles them.
#pragma once

#include "common.h"

namespace lgh {

// A bf16 weight matrix [n][k] kept as it came: rows padded to a multiple of 16, columns to a multiple of 64 (zeros).  Several
// matrices with the same input lie below one another (SEGMENTS, each starting at a multiple of 16 rows), so that one launch
// computes them all; a "paired" matrix (feed-forward gate | up) interleaves its two halves in blocks of 16 rows.
struct LinW {
  uint16_t* w = nullptr;
  uint32_t n = 0, k = 0;       // rows (all segments, padded to 16), columns that hold values
  uint32_t kp = 0;             // row stride in elements, multiple of 64
  bool paired = false;
  uint32_t np() const { return (n + 15) / 16 * 16; }
  size_t bytes() const { return (size_t)n * k * 2; }
};

// ---- residual form LGH_RESIDUAL_SANDWICH_DYT: h = dyt(x), h += conv(h), x += mult * dyt'(sublayer(h)); all of it per channel ----
struct DytW { const float *w = nullptr, *b = nullptr, *alpha = nullptr; };     // tanh(alpha v) * w + b
struct ConvW {                 // causal convolution, one filter per channel
  const float* w = nullptr;    // [width][taps], the last tap at the token itself
  float* hist = nullptr;       // [taps - 1][width]: the input at position p lies in row p % (taps - 1) until position p + taps - 1 replaces it
  uint32_t taps = 0;           // 0: no convolution
};
struct PostUpdate {            // a token's residual update and the next sublayer's input (decode: in the epilogue of the product before it)
  const float* x = nullptr;    // residual stream, updated to xout (may be the same vector)
  float* xout = nullptr;
  DytW post, next;
  ConvW conv;
  float* hout = nullptr;
  const int* pos = nullptr;    // device word: the token's position
  float mult = 1.0f;
  uint32_t width = 0;
};

// What a decode mat-vec does to its input vector before the product (every workgroup, in LDS)
enum LinPro : int {
  LP_COPY = 0,    // x
  LP_RESID = 1,   // x + mult * layer_norm(y) * nw, also written to xout (the new residual stream)
  LP_HEAD = 2,    // layer_norm of the same sum, times nw2 (final norm in front of the output projection)
  LP_MLSTM = 3,   // matrix-memory read-out: numerators / denominators, per-head RMS norm, norm weight, sigmoid gate
  LP_PRE = 4,     // v = x + mult * y (y may be absent), also written to xout; rms_norm(v) * (nw_add + nw2) * in_scale, also written to hout
  LP_SANDWICH = 5,// v = x + mult * layer_norm(y) * nw (y may be absent), also written to xout; layer_norm(v) * nw2
  LP_READ = 6,    // read-out of a matrix state: per-head RMS norm, one norm weight [vdim] for all heads, silu gate
};
// Which weights its rows come from
enum LinSrc : int {
  LS_PLAIN = 0,
  LS_TWO = 1,      // w, and below it w2 (plain rows, same input) -> out2; w may be absent
  LS_EXPERTS = 2,  // the top experts of `logits` (every workgroup ranks them), their gate | up pairs; the input is weighted by the expert's score
  LS_MOE_DOWN = 3, // input [shared | expert | expert ..]: a row is a row of w (shared, absent: kps = 0) followed by the same row of every chosen expert
};
enum LinAct : uint32_t { LA_GELU = 0, LA_SILU = 1, LA_CLAMPED = 2,     // act(gate) * up; LA_CLAMPED: clamped_glu_f
                        LA_RELU2 = 3 };                                  // unpaired rows: relu(v)^2
// how a token's experts are chosen (LGH_ROUTER_*)
struct RouteForm {
  uint32_t form = LGH_ROUTER_SIGMOID;
  uint32_t groups = 1, keep = 1, identity = 0;
  const float* correction = nullptr;   // [experts + identity]
};
struct LinMv {
  const uint16_t* w;
  uint32_t n, kp, k, paired;   // paired: 0 or 1
  float* out;                  // [n], paired: [n / 2] = act(gate) * up
  uint32_t act;                // LinAct
  const float* x;
  const float* y;              // LP_RESID / LP_HEAD: the pending sublayer output
  const float* nw;             // its norm weight
  const float* nw2;
  float* xout;
  float eps, mult, in_scale;
  float nw_add;                // LP_PRE
  float cap;                   // unpaired rows: cap * tanh(v / cap) (0: none)
  const float* bias;           // [n], unpaired rows (NULL: none)
  float* hout;                 // LP_PRE: the input vector (NULL: not kept)
  float limit;                 // LA_CLAMPED
  const float* num;            // LP_READ: [heads][ldo]; LP_MLSTM: [heads][ldo] numerators, column vdim = n . q, column vdim + 1 = exp(-m)
  const float* gate;
  uint32_t heads, vdim, ldo;
  const uint16_t* w2;          // LS_TWO: second matrix; LS_EXPERTS / LS_MOE_DOWN: the experts, one below the other
  float* out2;
  uint32_t n2;
  const float* logits;         // LS_EXPERTS: [experts] router logits
  uint32_t experts, top;
  int* sel;                    // [top] chosen experts: written by LS_EXPERTS, read by LS_MOE_DOWN
  uint64_t stride;             // elements between two experts
  RouteForm route;             // LS_EXPERTS (a form other than sigmoid scores weights the experts' outputs, with `logits` [experts + identity])
  float* selw;                 // [top] weights of the chosen: written by LS_EXPERTS; LS_MOE_DOWN: those of identity experts multiply id_x
  const float* id_x;           // LS_MOE_DOWN: what identity experts hand back (NULL: there are none)
  uint32_t kps, kpe;           // LS_MOE_DOWN: columns of the shared part and of an expert; LS_EXPERTS: an expert's outputs lie kpe apart
  PostUpdate post;             // post.xout set: rows are not stored but update the residual stream
};
bool route_ok(const RouteForm& f, uint32_t outputs, uint32_t top);   // LGH_ROUTER_SOFTMAX_GROUPS
hipError_t lin_mv_launch(int pro, const LinMv& a, hipStream_t st, int src = LS_PLAIN);
constexpr uint32_t kMaxExperts = 1024, kMaxTop = 64, kMaxRouted = 512;   // (the last: router outputs of LGH_ROUTER_SOFTMAX_GROUPS)
constexpr uint32_t kLinMvMaxK = 36864;   // input vectors live in LDS

// Matrix product of a block of tokens: out[m][n] = sum_k x[m][k] * w[n][k].  f32 = true: activations and products in 32-bit
// (f32 matrix cores), otherwise bf16 activations with f32 accumulation.
enum LinEpi : int {
  LE_F32 = 0,     // out: float [M][ldo]
  LE_ACT = 1,     // out: activation type [M][ldo]
  LE_GEGLU = 2,   // paired weights: gelu(gate) * up as activation type [M][ldo]
  LE_HEADS = 3,   // activation type, row n = head * hd + j of token m at out[(head * tcap + m) * ldo + j]
  LE_HEADS_T = 4, // activation type, transposed per head: out[(head * hrows + j) * ldo + m]
  LE_SWIGLU = 5,  // paired weights: silu(gate) * up as activation type [M][ldo]
  LE_RELU2 = 7,   // activation type, relu(v)^2
  LE_CLAMPED = 6, // grouped rows, paired weights: scale * clamped_glu_f(gate, up) as activation type [M][ldo]
};
// rows grouped by expert: row tile i takes rows tile_row[i] .. of the group tile_e[i] (-1: no tile), which ends at seg[group + 1]; that
// group's weights lie `stride` elements per group behind w
struct LinGroup {
  const int *seg = nullptr, *tile_e = nullptr, *tile_row = nullptr;
  const int* src = nullptr;        // row of x of every row (NULL: the same row)
  const float* scale = nullptr;    // factor of every row's input (LE_SWIGLU) or output (LE_CLAMPED)
  float limit = 0.0f;              // LE_CLAMPED
  uint64_t stride = 0;
  uint32_t tiles = 0, bm = 0;      // row tiles (upper bound) and their height
};
struct LinGemm {
  const uint16_t* w;
  const void* x;               // [M][ldx], columns k..kp of every row are zero
  void* out;
  uint32_t n, np, kp, ldx, ldo, M;
  uint32_t hd, hrows;          // LE_HEADS / LE_HEADS_T
  uint64_t tcap;
  const float* bias;           // LE_F32: [n] (NULL: none)
  float cap;                   // LE_F32: cap * tanh(v / cap) (0: none)
  LinGroup grp;
};
hipError_t lin_gemm_launch(int epi, bool f32, const LinGemm& a, hipStream_t st);
uint32_t lin_group_rows(uint32_t rows, uint32_t groups);   // height of a grouped product's row tiles for this many rows over this many groups
// upload: rows [row0, row0 + rows) of a bf16 matrix; mode 0 plain, 1 first half of a pair, 2 second half of a pair
hipError_t lin_pack_launch(const uint16_t* src, uint32_t rows, uint32_t k, uint16_t* dst, uint32_t kp, uint32_t row0, int mode, hipStream_t st);
// per head [dim][rank] -> [rank][dimp]
hipError_t lin_transpose_heads_launch(const uint16_t* src, uint32_t heads, uint32_t dim, uint32_t rank, uint16_t* dst, uint32_t dimp, hipStream_t st);

// ---- layered_misc.hip ----
struct EmbedArgs {
  const uint16_t* embed;       // [vocab][width] bf16
  const uint16_t* bigram;      // [buckets + 1][width] or NULL
  uint32_t width, buckets, ld; // ld: row stride of the embedding table
  uint64_t mul_prev, mul_cur;
  int* hist;                   // token of every position (the previous token is part of the sequence's state)
};
// post (may be NULL): also the first sublayer's input, LGH_RESIDUAL_SANDWICH_DYT
hipError_t layered_embed_launch(const EmbedArgs& a, int* state, float* x, const PostUpdate* post, hipStream_t st);
hipError_t layered_embed_block_launch(const EmbedArgs& a, const int* tokens, uint32_t pos0, uint32_t M, float* x, void* xa, uint32_t ldx, bool f32,
                                      hipStream_t st);
// x += mult * layer_norm(y) * w; also as activations
hipError_t resid_norm_launch(float* x, const float* y, uint32_t ldy, const float* w, float eps, float mult, uint32_t width, uint32_t M, void* xa,
                             uint32_t ldx, bool f32, hipStream_t st);
// decode without a consumer: xout = x + mult * layer_norm(y) * w
hipError_t resid_norm_out_launch(const float* x, const float* y, const float* w, float eps, float mult, uint32_t width, float* xout, hipStream_t st);
// rows[i] of x, layer-normed with w, as activations
hipError_t final_norm_rows_launch(const float* x, const int* rows, uint32_t n_rows, const float* w, float eps, uint32_t width, void* xa, uint32_t ldx,
                                  bool f32, hipStream_t st);
hipError_t final_dyt_rows_launch(const float* x, const int* rows, uint32_t n_rows, const DytW& n, uint32_t width, void* xa, uint32_t ldx, bool f32, hipStream_t st);

// LGH_RESIDUAL_SANDWICH_DYT over a block: v = x + mult * dyt(y), y = `y` (may be NULL) plus a token's rows of `pairs` in slot order;
// v -> xout (another buffer than x; NULL without a sublayer output: v = x), the next sublayer's input -> xa (NULL: none).  The inputs of
// the convolution at the block's last taps - 1 positions go to `tail` [taps - 1][width], row i = i positions before the last.
struct DytBlock {
  const float* x;
  float* xout;
  const float* y;
  uint32_t ldy;
  const float* pairs;          // [M * top][ldp], with slot[t * top + s] = the row of token t's s-th expert; NULL: none
  const int* slot;
  uint32_t ldp, top;
  DytW post, next;
  ConvW conv;
  float* tail;
  void* xa;
  uint32_t ldx, width, M, pos0;
  float mult;
};
hipError_t dyt_block_launch(const DytBlock& a, bool f32, hipStream_t st);
// after a block: tails [n_sub][taps - 1][width] -> histories [n_sub][taps - 1][width] (row of position p: p % (taps - 1))
hipError_t conv_store_launch(const float* tails, float* hists, uint32_t n_sub, uint32_t taps, uint32_t width, uint32_t pos0, uint32_t M, hipStream_t st);
// y[t] += a token's rows of `pairs` in slot order (a mixture in front of LGH_RESIDUAL_POST_LN); add = false: y[t] = the rows' sum
hipError_t pair_sum_launch(float* y, uint32_t ldy, const float* pairs, uint32_t ldp, const int* slot, uint32_t top, uint32_t width, uint32_t M, bool add, hipStream_t st);

// LGH_RESIDUAL_PRE_RMS over a block: x += mult * (y + a token's rows of `pairs` in slot order); a slot of -1 stands for selw * (the sublayer's
// input, still in xa).  rms_norm(x) * (1 + nw) -> xa (nw NULL: not wanted).  y and pairs may be NULL.
struct PreBlock {
  float* x;
  const float* y;
  const float* pairs;
  const int* slot;
  const float* selw;
  const float* nw;
  void* xa;
  uint32_t ldy, ldp, top, ldx, width, M;
  float eps, mult;
};
hipError_t pre_block_launch(const PreBlock& a, bool f32, hipStream_t st);
// LGH_RESIDUAL_SANDWICH_LN over a block: x += mult * layer_norm(y) * pw (y NULL: not yet); layer_norm(x) * nw -> xa (nw NULL: not wanted)
struct LnBlock {
  float* x;
  const float *y, *pw, *nw;
  void* xa;
  uint32_t ldy, ldx, width, M;
  float eps, mult;
};
hipError_t ln_block_launch(const LnBlock& a, bool f32, hipStream_t st);
// rms_norm of n columns of every row * w, as activations (columns n .. ldx are not touched)
hipError_t rms_cols_launch(const float* x, uint32_t ld, const float* w, float eps, uint32_t n, uint32_t M, void* xa, uint32_t ldx, bool f32, hipStream_t st);
hipError_t vec_mul_launch(float* x, const float* y, uint32_t n, hipStream_t st);   // x *= y
// decode without a consumer: xout = x + mult * y
hipError_t resid_add_launch(const float* x, const float* y, float mult, uint32_t width, float* xout, hipStream_t st);
hipError_t final_rms_rows_launch(const float* x, const int* rows, uint32_t n_rows, const float* w, float eps, float scale, uint32_t width, void* xa, uint32_t ldx,
                                 bool f32, hipStream_t st);

// ---- moe_route.hip: a block's tokens to their experts ----
struct MoeRoute {
  const void* x;               // [M][ldx]
  const uint16_t* router;      // [experts][kp]
  uint32_t ldx, kp, M, experts, top, bm;
  int* sel;                    // [M * top] chosen experts, largest score first
  float* w;                    // [M * top] their scores
  int *seg, *tile_e, *tile_row;   // LinGroup, row tiles of bm rows
  int *slot;                   // [M * top]: row of the pair
  int *src;                    // [M * top]: token of the row
  float* roww;                 // [M * top]: score of the row
  uint32_t tiles;              // entries of tile_e / tile_row
  RouteForm route;             // (the chosen ones from `experts` on are identity experts: their slot is -1)
};
uint32_t moe_max_tiles(uint32_t rows, uint32_t experts, uint32_t bm);
hipError_t moe_route_launch(const MoeRoute& a, bool f32, hipStream_t st);   // router product, scores, groups

// ---- tied_attention.hip: grouped heads, values = keys before their norm ----
struct TiedShape {
  uint32_t heads, kv_heads, dim, dp;   // dp: row stride of the cache, multiple of 64
  uint32_t off_q, off_k, ldcat;
  uint32_t window, keep;               // i sees j <= i with i - j < window or j < keep
  uint64_t rows;                       // cache rows per key head, multiple of 64
  float scale, cap, eps;               // cap 0: none
};
struct TiedBufs {
  const float* cat;                    // [M][ldcat]
  const float *qn, *kn, *temp, *sink;  // norm weights [heads * dim], [kv_heads * dim]; per head
  void* cache;                         // [kv_heads][rows][dp]: keys as projected
  float* kinv;                         // [rows]: 1 / rms over all of a position's keys
  void* q;                             // blocks: [heads][Mcap][dp], norm weights (of the key too), temp and scale in them
  uint32_t Mcap;
  float *part_ml, *part_acc;           // [split][M * heads][2], [split][M * heads][dim]
};
constexpr uint32_t kTiedMaxSplits = 128, kTiedShort = 16, kTiedMaxDim = 256;   // portions up to kTiedShort tokens take the decode kernel
uint32_t tied_keys_per_round(const TiedShape& s, bool f32);   // keys of a workgroup per round of the decode kernel
uint32_t tied_splits(const TiedShape& s, uint32_t max_seq, uint32_t M, bool f32, uint32_t forced);
// one token (own = true: its key is taken from cat and written to the cache) or M tokens whose keys are in the cache
hipError_t tied_attn_launch(const TiedShape& s, const TiedBufs& b, const int* pos_ptr, uint32_t pos0, uint32_t M, bool own, uint32_t n_splits, bool f32, hipStream_t st);
hipError_t tied_merge_launch(const TiedShape& s, const TiedBufs& b, const int* pos_ptr, uint32_t pos0, uint32_t M, uint32_t n_splits, bool f32, void* out, uint32_t ldo,
                             bool out_f32, hipStream_t st);
hipError_t tied_prep_launch(const TiedShape& s, const TiedBufs& b, uint32_t pos0, uint32_t M, bool f32, hipStream_t st);
hipError_t tied_flash_launch(const TiedShape& s, const TiedBufs& b, uint32_t pos0, uint32_t M, bool f32, void* out, uint32_t ldo, hipStream_t st);

// ---- gla.hip: gated linear attention, S_t = diag(alpha_t) S_(t-1) + k_t v_t^T per head, out S_t^T q_t ----
struct GlaShape {
  uint32_t heads, dim, vdim, rank;     // rank: inner size of the decay's projection
  uint32_t lds, ldo;                   // row strides: state [head][dim][lds], outputs before their norm [M][heads][ldo]
  uint32_t off_q, off_k, off_v, off_g, off_a, ldcat;
  uint32_t a2_ld;
  float tau, eps, out_scale;
};
struct GlaBufs {
  const float* cat;                    // [M][ldcat], blocks: + kMlstmRowSlack
  const uint16_t* a2;                  // [heads * dim][a2_ld]
  const float *a2b, *norm;             // [heads * dim], [vdim]
  float* S;
  float* num;                          // [M][heads][ldo]
  float* qk;                           // blocks: [Mcap][2 * heads * dim] decayed queries | keys, + kMlstmRowSlack
  float* dec;                          // blocks: [chunk][heads * dim] a chunk's whole decay, + kMlstmRowSlack
  float* a;                            // blocks: [chunk][heads][64][64] decayed scores
  uint32_t Mcap;
};
hipError_t gla_step_launch(const GlaShape& s, const GlaBufs& b, const int* pos_ptr, uint32_t pos0, hipStream_t st);
hipError_t gla_block_launch(const GlaShape& s, const GlaBufs& b, uint32_t pos0, uint32_t M, hipStream_t st);
// per-head RMS norm, norm weight, silu gate, out_scale -> columns of out
hipError_t gla_out_launch(const GlaShape& s, const GlaBufs& b, uint32_t M, void* out, uint32_t ldo, bool f32, hipStream_t st);

// ---- gated_attention.hip: grouped heads with values of their own; norms, gate, chunks, window and sink as the layer has them ----
struct GattnShape {
  uint32_t heads, kv_heads, dim, vdim, dp, vp;   // dp, vp: row strides of the caches, multiples of 64
  uint32_t off_q, off_k, off_v, off_g, ldcat;
  uint32_t chunk, window;              // i sees j <= i with j / chunk == i / chunk and i - j < window
  uint32_t gated, sink;                // 0 or 1: outputs times sigmoid(cat + off_g); the softmax's denominator has one more term, exp(0)
  uint32_t rot_n;                      // leading values of a head that are rotated
  uint64_t rows;                       // cache rows per key head, multiple of 64
  float scale, eps, out_scale;
};
struct GattnBufs {
  const float* cat;                    // [M][ldcat]
  const float *qn, *kn, *cs;           // norm weights [dim] (NULL: queries and keys are not normed); [max_seq][rot_n / 2][2]
  bool shared;                         // the keys and values are another layer's: nothing is written to the caches
  void *kc, *vc;                       // [kv_heads][rows][dp | vp]: keys normed and rotated, values
  void* q;                             // blocks: [heads][Mcap][dp]
  uint32_t Mcap;
  float *part_ml, *part_acc;           // [split][M * heads][2], [split][M * heads][vdim]
};
constexpr uint32_t kGattnShort = 16, kGattnMaxDim = 512, kGattnFlashDim = 256;
uint32_t gattn_splits(const GattnShape& s, uint32_t max_seq, uint32_t M, bool f32, uint32_t forced);
// one token (own = true: its key and value are taken from cat and written to the cache) or M tokens whose rows are in the cache; gla (may be
// NULL, own only): a step of gated linear attention in the same launch
hipError_t gattn_attn_launch(const GattnShape& s, const GattnBufs& b, const GlaShape* gs, const GlaBufs* gb, const int* pos_ptr, uint32_t pos0, uint32_t M, bool own,
                             uint32_t n_splits, bool f32, hipStream_t st);
// the shares put together, gated -> out; gla: its read-out behind them, from column gla_col on (decode)
hipError_t gattn_merge_launch(const GattnShape& s, const GattnBufs& b, const GlaShape* gs, const GlaBufs* gb, uint32_t gla_col, const int* pos_ptr, uint32_t pos0,
                              uint32_t M, uint32_t n_splits, bool f32, void* out, uint32_t ldo, bool out_f32, hipStream_t st);
hipError_t gattn_prep_launch(const GattnShape& s, const GattnBufs& b, uint32_t pos0, uint32_t M, bool f32, hipStream_t st);
hipError_t gattn_flash_launch(const GattnShape& s, const GattnBufs& b, uint32_t pos0, uint32_t M, bool f32, void* out, uint32_t ldo, hipStream_t st);

// ---- delta.hip: gated delta rule, S_t = g_t S_(t-1) + k_t u_t^T with u_t = beta_t (v_t - g_t S_(t-1)^T k_t) per head, out S_t^T q_t ----
struct DeltaShape {
  uint32_t heads, kv_heads, dim, vdim, taps;
  uint32_t dk, lv;                     // dim, vdim up to 16: row strides of queries and keys; of the state [head][dk][lv], values and outputs
  uint32_t off_q, off_k, off_v, off_g, off_b, off_a, ldcat;
  uint32_t cols;                       // leading columns of cat that pass the convolution (queries, keys, values)
  float eps;
};
struct DeltaBufs {
  const float* cat;                    // [M][ldcat]
  const float* conv;                   // [cols][taps], the last tap at the token itself
  const float *a_log, *dt, *norm;      // [heads], [heads], [vdim]
  float* S;
  float* hist;                         // [taps][cols]: the convolution's input at position p lies in row p % taps
  float* num;                          // [M][heads][lv] outputs before their norm; blocks: whole chunks of 64 tokens
  // blocks, whole chunks of 64 tokens (zeros behind the last token and in the padding)
  float *q, *k;                        // [Mcap][kv_heads][dk] unit queries (times dim^-1/2) and keys
  float *v, *u;                        // [Mcap][heads][lv] values; what a chunk writes from an empty state
  float *w, *p;                        // [Mcap][heads][dk] what the state before the chunk takes off u; what it adds to the outputs
  float *wge, *cd;                     // [heads][Mcap] decay from a token to its chunk's end; [heads][Mcap / 64] a chunk's decay
  uint32_t Mcap;
};
constexpr uint32_t kDeltaBlockDim = 512;     // larger heads take blocks token by token
hipError_t delta_step_launch(const DeltaShape& s, const DeltaBufs& b, const int* pos_ptr, uint32_t pos0, hipStream_t st);
hipError_t delta_block_launch(const DeltaShape& s, const DeltaBufs& b, uint32_t pos0, uint32_t M, hipStream_t st);
// read-out of a block (per-head RMS norm, norm weight, silu gate), and what the sequence keeps of the convolution's inputs
hipError_t delta_out_launch(const DeltaShape& s, const DeltaBufs& b, uint32_t pos0, uint32_t M, void* out, uint32_t ldo, bool f32, hipStream_t st);

// ---- glru.hip: S_t = a_t S_(t-1) + sqrt(1 - a_t^2) i_t u_t per channel ----
struct GlruShape {
  uint32_t width, blocks, bs, taps;    // bs: channels of a diagonal block
  uint32_t off_y, off_x, ldcat;
  uint32_t gate_rows, gate_kp;         // gates [block][gate_rows][gate_kp]: r and i interleaved in blocks of 16 rows
};
struct GlruBufs {
  const float* cat;                    // [M][ldcat]
  const float *conv, *conv_b;          // [width][taps], [width]
  const uint16_t* gates;
  const float *rb, *ib, *lam;          // [width]
  float* S;                            // [width]
  float* hist;                         // [taps][width]: the convolution's input at position p lies in row p % taps
  float *a, *x;                        // blocks: [M][width] factors and inputs of the recurrence
  float* sum;                          // blocks: [chunk][width][2] a chunk of 64 tokens as one factor and one input
  float* s0;                           // blocks: [width] state before the block
};
hipError_t glru_step_launch(const GlruShape& s, const GlruBufs& b, const int* pos_ptr, float* out, hipStream_t st);
hipError_t glru_block_launch(const GlruShape& s, const GlruBufs& b, uint32_t pos0, uint32_t M, bool f32, void* out, uint32_t ldo, hipStream_t st);

// ---- latent_attention.hip ----
struct LatentShape {
  uint32_t heads, dim, rot_dim, rot_n, vdim, rank;
  uint32_t ldc;                // elements of a cache row: [latent rank | rotated key part rot_dim | zeros], multiple of 64
  uint32_t dimp, rankp;        // row strides of the transposed key expansion [head][rank][dimp] and the value expansion [head * vdim][rankp]
  uint32_t off_q, off_dkv, off_g, ldcat;   // where a token's projections lie in its row of the fused product (off_q: queries, or their latent)
  uint32_t ldq;                // row stride of the queries
  uint32_t window;             // i sees j <= i with i - j < window
  uint32_t halves, gate_values;   // 0 or 1: pairs (i, i + rot_n / 2) instead of (2i, 2i + 1); a gate per value instead of per head
  float scale, eps;
};
struct LatentBufs {
  const float* cat;            // [M][ldcat]
  const float* q;              // [M][ldq]: queries, head by head [dim | rot_dim]
  const float* dkv_norm;       // [rank]
  const float* cs;             // [max_seq][rot_n / 2][2]
  const uint16_t *uk_t, *uv;
  void* cache;                 // [max_seq][ldc]
  void* qa;                    // [M * heads][ldc]: absorbed queries
  float *part_ml, *part_acc;   // [split][M * heads][2], [split][M * heads][rank]
};
constexpr uint32_t kLatMaxSplits = 128;
constexpr uint32_t kLatAbsorbRows = 1024;   // (token, head) rows the absorbed path's buffers hold
// pos_ptr (device) or pos0: position of the first of the M tokens
hipError_t latent_prep_launch(const LatentShape& s, const LatentBufs& b, const int* pos_ptr, uint32_t pos0, uint32_t M, bool f32, hipStream_t st);
hipError_t latent_attn_launch(const LatentShape& s, const LatentBufs& b, const int* pos_ptr, uint32_t pos0, uint32_t M, uint32_t n_splits, bool f32,
                              hipStream_t st);
// merges the splits, expands the latent to the value and applies the head gate -> out [M][ldo] (f32 vector in decode, activations otherwise)
hipError_t latent_out_launch(const LatentShape& s, const LatentBufs& b, const int* pos_ptr, uint32_t pos0, uint32_t M, uint32_t n_splits, void* out, uint32_t ldo, bool out_f32, hipStream_t st);
bool latent_fits(const LatentShape& s, bool f32);   // the absorbed kernel's tiles fit LDS
// expanded path (long prompts): keys and values per head, from position `base` on
struct LatentFlash {
  void* q;                     // [heads][Mcap][dq]
  void* k;                     // [heads][Tcap][dq]
  void* vt;                    // [heads][dvp][Tcap]
  uint32_t dq, dvp, Mcap;
  uint32_t base;               // a multiple of 64, no position before it is visible
  uint64_t Tcap;
};
uint32_t latent_key_start(const LatentShape& s, uint32_t i);   // the first key that position i sees
bool latent_flash_shape(const LatentShape& s, uint32_t* dq, uint32_t* dvp);
hipError_t latent_flash_prep_launch(const LatentShape& s, const LatentBufs& b, const LatentFlash& f, uint32_t pos0, uint32_t M, bool f32, hipStream_t st);
hipError_t latent_flash_launch(const LatentShape& s, const LatentBufs& b, const LatentFlash& f, uint32_t pos0, uint32_t M, bool f32, void* out,
                               uint32_t ldo, hipStream_t st);

// ---- mlstm.hip ----
struct MlstmShape {
  uint32_t heads, dim, vdim;
  uint32_t lds;                // row stride of the state [head][dim][lds]: columns 0..vdim-1 = S, column vdim = n
  uint32_t ldo;                // row stride of the numerators [M][heads][ldo]
  uint32_t off_q, off_k, off_v, off_g, off_i, off_f, ldcat;
  uint32_t ldqk;               // row stride of the queries and keys of a block (qk)
  float cap, eps;
};
struct MlstmBufs {
  const float* cat;            // [M][ldcat], blocks: + kMlstmRowSlack
  const float *bi, *bf;        // [heads]
  const float* norm;           // [heads * vdim]
  float* S;
  double* m;                   // [2][heads]: the running maximum before position p lies in half p & 1
  float* num;                  // [M][heads][ldo]
  double *u, *mx;              // blocks: [heads][Mcap]
  float *dec, *wgt, *cdec;     // blocks: factors of the state kernel, [heads][Mcap] and [heads][chunks]
  float* nk;                   // blocks: [chunk][heads][dim]: a chunk's contribution to n, then n before the chunk
  float* a;                    // blocks: [chunk][heads][64][64] decayed scores
  const float* qk;             // blocks: queries and keys (off_q, off_k; rows of ldqk)
  const float* rowdec;         // mlstm_state_launch with a decay per state row: [chunk][heads * dim]
  uint32_t Mcap;
};
constexpr uint32_t kMlstmBlockDim = 512;      // larger heads take blocks token by token
constexpr uint32_t kMlstmRowSlack = 2048;   // floats the block kernels may read behind the last row of cat (never used)
hipError_t mlstm_step_launch(const MlstmShape& s, const MlstmBufs& b, const int* pos_ptr, hipStream_t st, uint32_t pos0 = 0);   // pos_ptr or pos0
hipError_t mlstm_block_launch(const MlstmShape& s, const MlstmBufs& b, uint32_t pos0, uint32_t M, hipStream_t st);
// a block's recurrence over its chunks alone; rowdec set: queries and keys carry their decays, every state row has its own decay per chunk
hipError_t mlstm_state_launch(const MlstmShape& s, const MlstmBufs& b, uint32_t pos0, uint32_t M, hipStream_t st);
hipError_t mlstm_out_launch(const MlstmShape& s, const MlstmBufs& b, uint32_t M, void* out, uint32_t ldo, bool f32, hipStream_t st);

}  // namespace lgh
