// layered.hip — models whose layers are described one by one (lgh_create_layered): weight store, cache rows and recurrent states, the
// decode launch sequence (captured in the engine's token graphs) and the block path for prompt portions.
//
// Decode, per token (every residual update rides in the prologue of the product that reads it):
//   latent attention   fused q | latent | gate product -> queries absorbed, cache row written -> split attention -> merge + value
//                      expansion + gate -> output product
//   mLSTM              fused q | k | v | gates product -> recurrence step -> output product (read-out norm and gate in its prologue)
//   tied attention     fused q | k product -> split attention (norms of q and k in its prologue, cache row written) -> merge -> output product
//   gated attention    fused q | k | v | gate product -> split attention (norms and rotation in its prologue, cache rows written) -> merge + gate ->
//                      output product; a gated linear attention beside it steps and is read out in the same launches, one output product for both
//   grouped attention  the same without norms and gate; a layer that reads another layer's cache rows projects queries only
//   latent attention with a query latent: fused query latent | latent | gate product -> query product (the latent's norm in its prologue) -> as above
//   delta rule         fused q | k | v | gate, step and decay product -> convolution and state step -> output product (read-out norm and gate in its prologue)
//   linear recurrence  fused y | x product -> convolution, gates and recurrence step -> output product
//   feed-forward       gate | up product with gelu * in its epilogue (or up product with the squared relu) -> down product
//   mixture            shared gate | up + router product -> the chosen experts' gate | up (every workgroup ranks the scores) -> one down
//                      product over [shared | experts]
// With norms in front of the sublayers (LGH_RESIDUAL_PRE_RMS) the prologue of the product that reads the stream updates and norms it.
// With layer norms on both sides (LGH_RESIDUAL_SANDWICH_LN) it norms the sublayer's output, updates the stream and norms that.
// With squashing norms (LGH_RESIDUAL_SANDWICH_DYT) everything between two sublayers is per channel: it rides in the EPILOGUE of the
// product that finishes a channel, and no norm is computed more than once.
// A sequence's state: the cache rows, the matrix states (and running maxima), the linear recurrences, the convolutions' last inputs, and the last token
// (pair embedding), kept as a token history by position; a position of 0 makes every kernel ignore what is stored, so lgh_reset stays O(1).
#include <algorithm>
#include <cmath>
#include <map>

#include "engine.h"
#include "layered.h"

using namespace lgh;

namespace lgh {

constexpr uint32_t kBlockTokens = 2048;    // tokens per pass of the block path
constexpr uint32_t kLogitRows = 128;       // wanted rows per output product
constexpr uint32_t kMaxConvTaps = 64;
constexpr uint32_t kMaxRecTaps = 64;

struct LayeredLayer {
  lgh_layer_desc d{};
  LinW in, out, gu, down, uk, uv;          // mixer inputs (one product), mixer output, gate | up, down (mixture: of the shared expert), latent expansions
  LinW router, egu, edown;                 // mixture: router, the experts' gate | up and down, `egu_rows` and `edown_rows` rows each
  uint32_t egu_rows = 0, edown_rows = 0;
  float *qn = nullptr, *kn = nullptr, *temp = nullptr, *sink = nullptr, *kinv = nullptr;
  uint32_t splits = 1;
  TiedShape ts{};
  GattnShape gs{};
  GlaShape as{};
  GlruShape rs{};
  DeltaShape des{};
  LinW uq;                                 // latent attention: the queries' second projection
  float *dq_norm = nullptr, *a_log = nullptr, *dt = nullptr, *out_bias = nullptr;
  float *post1 = nullptr, *post2 = nullptr, *ls1 = nullptr, *ls2 = nullptr;   // LGH_RESIDUAL_SANDWICH_LN: norms behind the sublayers (times ls, from finalize on)
  LinW a2, gates;                          // linear attention: the decay's second factor; linear recurrence: its gates' diagonal blocks
  float *in_bias = nullptr, *a2b = nullptr, *gnorm = nullptr, *conv = nullptr, *conv_b = nullptr, *rb = nullptr, *ib = nullptr, *lam = nullptr, *correction = nullptr;
  float *rS = nullptr, *rhist = nullptr;
  void* vcache = nullptr;
  uint32_t gla_col = 0;                    // where the linear attention's values lie in the output product's input
  uint16_t* uk_t = nullptr;
  float *norm1 = nullptr, *norm2 = nullptr, *dkv_norm = nullptr, *mnorm = nullptr, *bi = nullptr, *bf = nullptr, *cs = nullptr;
  void* cache = nullptr;
  float* S = nullptr;
  double* m = nullptr;
  LatentShape ls{};
  MlstmShape ms{};
  bool latent() const { return d.mixer == LGH_MIXER_LATENT_ATTENTION; }
  bool mlstm() const { return d.mixer == LGH_MIXER_MLSTM; }
  bool tied() const { return d.mixer == LGH_MIXER_TIED_ATTENTION; }
  bool grouped() const { return d.mixer == LGH_MIXER_GROUPED_ATTENTION; }
  bool gattn() const { return d.mixer == LGH_MIXER_GATED_ATTENTION || d.mixer == LGH_MIXER_PARALLEL || grouped(); }
  bool delta() const { return d.mixer == LGH_MIXER_DELTA; }
  bool gla() const { return d.mixer == LGH_MIXER_GLA || d.mixer == LGH_MIXER_PARALLEL; }
  bool glru() const { return d.mixer == LGH_MIXER_GLRU; }
  bool rotated() const { return latent() || gattn(); }
  bool moe() const { return d.ff_kind == LGH_FF_MOE; }
  RouteForm route() const {
    RouteForm r;
    r.form = d.router_form;
    if (r.form == LGH_ROUTER_SOFTMAX_GROUPS) { r.groups = d.groups; r.keep = d.keep_groups; r.identity = d.identity; r.correction = correction; }
    return r;
  }
  uint32_t act_cols() const { return moe() ? down.kp + d.top * edown.kp : down.kp; }   // inputs of the down product
};

struct LayeredNorm { float *w = nullptr, *b = nullptr, *alpha = nullptr; };
struct LayeredSub {                        // LGH_RESIDUAL_SANDWICH_DYT: what surrounds a sublayer
  LayeredNorm pre, post;
  float* conv = nullptr;
};

struct LayeredSlot {                       // where a named tensor goes
  LinW* mat = nullptr;
  uint32_t row0 = 0, n = 0, k = 0;
  int mode = 0;
  float** vec = nullptr;
  uint32_t off = 0, total = 0;             // vec: this tensor's place in a vector of `total` values (0: the tensor is the vector)
  uint32_t col0 = 0, parts = 1;            // mat: first column; equal parts, each of `stride` rows
  uint32_t stride = 0;
  uint16_t** raw = nullptr;
  LayeredLayer* transpose = nullptr;
  bool done = false;
};

struct LayeredModel {
  lgh_layered_desc d{};
  std::vector<LayeredLayer> layers;
  std::map<std::string, LayeredSlot> slots;
  uint16_t *embed = nullptr, *bigram = nullptr;
  LinW head;
  float* final_norm = nullptr;
  int* tokens = nullptr;                   // token of every position
  bool f32 = false, recurrent = false;
  uint32_t forced_splits = 0;              // LGH_FLAG_ATTN_SPLITS_SHIFT
  uint32_t n_sub = 0, n_splits = 1;
  // LGH_RESIDUAL_SANDWICH_DYT
  std::vector<LayeredSub> subs;
  LayeredNorm final_dyt;
  float *h = nullptr, *hist = nullptr, *tails = nullptr;   // a sublayer's input (decode); the convolutions' histories and a block's last inputs
  bool ln2() const { return d.residual == LGH_RESIDUAL_SANDWICH_LN; }
  bool dyt() const { return d.residual == LGH_RESIDUAL_SANDWICH_DYT; }
  bool pre() const { return d.residual == LGH_RESIDUAL_PRE_RMS; }
  size_t hist_floats() const { return d.conv_taps > 1 ? (size_t)n_sub * (d.conv_taps - 1) * d.width : 0; }
  // mixtures
  float* rlogits = nullptr;
  int* sel = nullptr;
  float* selw = nullptr;
  uint32_t max_experts = 0, max_top = 0, max_pair_act = 0;   // (the last: top * columns of an expert)
  float *bpair = nullptr, *bselw = nullptr, *broww = nullptr;
  int *bsel = nullptr, *bseg = nullptr, *btile_e = nullptr, *btile_row = nullptr, *bslot = nullptr, *bsrc = nullptr;
  void* bpact = nullptr;
  // tied and gated attention's queries of a block
  uint32_t max_tied_q = 0;                 // heads * row
  size_t max_tied_rows = 0, max_tied_acc = 0;   // partial sums: (token, head) rows * splits, and times the head size
  void* btq = nullptr;
  // decode
  float *x[2] = {nullptr, nullptr}, *y = nullptr, *cat = nullptr, *ao = nullptr, *act = nullptr, *num = nullptr, *part_ml = nullptr, *part_acc = nullptr;
  void* qa = nullptr;
  float* lq = nullptr;                     // latent attention with a query latent: a token's queries
  uint32_t max_lq = 0, max_qrank = 0;
  uint32_t max_cat = 0, max_ao = 0, max_act = 0, max_num = 0;
  // blocks
  bool blk_ready = false;
  uint32_t blk = 0;
  float *bx2 = nullptr;                    // LGH_RESIDUAL_SANDWICH_DYT: the stream's second buffer
  float *bx = nullptr, *by = nullptr, *bcat = nullptr, *bnum = nullptr, *ba = nullptr, *blogits = nullptr;
  double *bu = nullptr, *bmx = nullptr;
  float *brec = nullptr, *brsum = nullptr, *bqk = nullptr, *bgdec = nullptr;   // linear recurrence: factors | inputs, tiles; linear attention
  uint32_t max_rec = 0, max_gla = 0;       // channels of a recurrence; heads * dim of a linear attention
  float *bdec = nullptr, *bwgt = nullptr, *bcdec = nullptr, *bnk = nullptr;
  void *bxa = nullptr, *bao = nullptr, *bact = nullptr, *bla = nullptr;
  int *btok = nullptr, *brows = nullptr;
  float* blq = nullptr;                    // queries made from their latent
  void* blqa = nullptr;                    // that latent, normed
  uint32_t max_dqk = 0, max_dw = 0, max_dv = 0, max_dheads = 0;   // delta rules: kv_heads * dk, heads * dk, heads * lv, heads
  float *bdq = nullptr, *bdk = nullptr, *bdv = nullptr, *bdu = nullptr, *bdw = nullptr, *bdp = nullptr, *bdwge = nullptr, *bdcd = nullptr;
  // expanded attention (grown with the context)
  LatentFlash fl{};
  size_t fl_q_bytes = 0, fl_k_bytes = 0, fl_v_bytes = 0;
  // layer tap
  bool tap = false;
  float* tap_buf = nullptr;
  uint32_t tap_tokens = 0;
  uint32_t el() const { return f32 ? 4 : 2; }
};

}  // namespace lgh

static uint32_t up(uint32_t v, uint32_t a) { return (v + a - 1) / a * a; }

#define L_TRY(c, status, expr)                                                                                    \
  do {                                                                                                            \
    hipError_t e__ = (expr);                                                                                      \
    if (e__ != hipSuccess) return fail((c), (status), std::string(#expr) + ": " + hipGetErrorString(e__));        \
  } while (0)

void layered_destroy(lgh_ctx* c) {
  delete c->lm;
  c->lm = nullptr;
}
bool layered_recurrent(const lgh_ctx* c) { return c->lm->recurrent || c->lm->d.conv_taps > 1; }
bool layered_has_blocks(const lgh_ctx* c) { return !(c->d.flags & LGH_FLAG_EXACT_PREFILL); }

// What the kernels can hold, checked before anything is allocated
static int layered_check(const lgh_layered_desc& d, const lgh_layer_desc* L, std::string& why) {
  if (!d.width || !d.vocab_size || !d.num_layers || !d.max_seq_len) { why = "a model dimension is zero"; return LGH_INVALID_ARGUMENT; }
  if (d.compute > LGH_COMPUTE_F32) { why = "unknown compute type"; return LGH_INVALID_ARGUMENT; }
  if (!(d.norm_eps >= 0.0) || !std::isfinite(d.residual_mult)) { why = "norm_eps / residual_mult"; return LGH_INVALID_ARGUMENT; }
  if (up(d.width, 64) > 32768) { why = "width above 32768"; return LGH_UNSUPPORTED; }
  if (d.tied_head > 1 || !std::isfinite(d.logit_scale)) { why = "output projection"; return LGH_INVALID_ARGUMENT; }
  if (d.logit_scale != 0.0 && d.logit_scale != 1.0 && d.residual != LGH_RESIDUAL_PRE_RMS) { why = "a factor on the logits"; return LGH_UNSUPPORTED; }
  if (!(d.logit_cap >= 0.0) || !std::isfinite(d.logit_cap)) { why = "a cap of the logits"; return LGH_INVALID_ARGUMENT; }
  if (d.residual > LGH_RESIDUAL_SANDWICH_LN) { why = "unknown residual form"; return LGH_UNSUPPORTED; }
  if (d.conv_taps > kMaxConvTaps || (d.conv_taps && d.residual != LGH_RESIDUAL_SANDWICH_DYT)) { why = "convolution taps"; return LGH_UNSUPPORTED; }
  for (uint32_t i = 0; i < d.num_layers; i++) {
    const lgh_layer_desc& l = L[i];
    const std::string at = "layer " + std::to_string(i) + ": ";
    if (l.struct_size != sizeof(lgh_layer_desc)) { why = at + "descriptor size"; return LGH_INVALID_ARGUMENT; }
    if (l.mixer != LGH_MIXER_GLA && (!l.heads || !l.dim || !l.vdim)) { why = at + "a mixer dimension is zero"; return LGH_INVALID_ARGUMENT; }
    if (l.ff_kind > LGH_FF_RELU2 || (l.ff_kind && !l.ff)) { why = at + "feed-forward"; return LGH_INVALID_ARGUMENT; }
    if (l.ff_kind == LGH_FF_MOE && d.residual == LGH_RESIDUAL_SANDWICH_LN) { why = at + "mixtures between layer norms"; return LGH_UNSUPPORTED; }
    if (l.ff_kind == LGH_FF_MOE) {
      if (l.router_form > LGH_ROUTER_SOFTMAX_GROUPS || l.expert_form > LGH_EXPERT_CLAMPED) { why = at + "router or expert form"; return LGH_UNSUPPORTED; }
      const bool grp = l.router_form == LGH_ROUTER_SOFTMAX_GROUPS;
      if (!grp && l.identity) { why = at + "identity experts"; return LGH_UNSUPPORTED; }
      if (!l.experts || !l.top || l.top > l.experts + l.identity) { why = at + "experts"; return LGH_INVALID_ARGUMENT; }
      if (grp) {
        const uint32_t n = l.experts + l.identity;
        if (n > kMaxRouted) { why = at + "more than " + std::to_string(kMaxRouted) + " router outputs"; return LGH_UNSUPPORTED; }
        if (!l.groups || n % l.groups || !l.keep_groups || l.keep_groups > l.groups || l.keep_groups * (n / l.groups) < l.top) { why = at + "groups of experts"; return LGH_INVALID_ARGUMENT; }
        if (l.identity && d.residual != LGH_RESIDUAL_PRE_RMS) { why = at + "identity experts need a norm in front of the sublayer"; return LGH_UNSUPPORTED; }
        if (l.expert_form != LGH_EXPERT_CLAMPED || l.shared_ff) { why = at + "softmax routing takes clamped experts, none of them shared"; return LGH_UNSUPPORTED; }
      } else if (l.expert_form != LGH_EXPERT_SWIGLU) { why = at + "clamped experts take softmax routing"; return LGH_UNSUPPORTED; }
      if (l.experts > kMaxExperts || l.top > kMaxTop) { why = at + "more than " + std::to_string(kMaxExperts) + " experts or " + std::to_string(kMaxTop) + " per token"; return LGH_UNSUPPORTED; }
      if ((uint64_t)up(l.shared_ff, 64) + (uint64_t)l.top * up(l.ff, 64) > kLinMvMaxK) { why = at + "a token's experts together above " + std::to_string(kLinMvMaxK); return LGH_UNSUPPORTED; }
    } else if (l.ff_kind && up(l.ff, 64) > kLinMvMaxK) { why = at + "feed-forward above " + std::to_string(kLinMvMaxK); return LGH_UNSUPPORTED; }
    const bool gr = l.mixer == LGH_MIXER_GROUPED_ATTENTION, ga = l.mixer == LGH_MIXER_GATED_ATTENTION || l.mixer == LGH_MIXER_PARALLEL || gr, la = l.mixer == LGH_MIXER_GLA || l.mixer == LGH_MIXER_PARALLEL;
    if ((uint64_t)(l.mixer == LGH_MIXER_GLA ? 0 : up(l.heads * l.vdim, 64)) + (la ? up(l.gla_heads * l.gla_vdim, 64) : 0) > kLinMvMaxK) { why = at + "heads * vdim above " + std::to_string(kLinMvMaxK); return LGH_UNSUPPORTED; }
    if (l.mixer == LGH_MIXER_LATENT_ATTENTION) {
      if (!l.kv_rank || l.rot_dims > l.rot_dim || l.rot_dims % 2) { why = at + "latent attention sizes"; return LGH_INVALID_ARGUMENT; }
      if (l.rot_dims && !(l.rot_base > 0.0)) { why = at + "rotation base"; return LGH_INVALID_ARGUMENT; }
      if (l.rot_form > LGH_ROT_HALVES || l.gate_form > LGH_GATE_VALUES) { why = at + "rotation or gate form"; return LGH_UNSUPPORTED; }
      if (up(l.q_rank, 64) > kLinMvMaxK) { why = at + "query latent above " + std::to_string(kLinMvMaxK); return LGH_UNSUPPORTED; }
      LatentShape s{};
      s.rank = l.kv_rank;
      s.ldc = up(l.kv_rank + l.rot_dim, 64);
      if (l.heads > kLatAbsorbRows || !latent_fits(s, d.compute == LGH_COMPUTE_F32)) { why = at + "latent rows too large for LDS"; return LGH_UNSUPPORTED; }
    } else if (l.mixer == LGH_MIXER_TIED_ATTENTION) {
      if (!l.kv_heads || l.heads % l.kv_heads || l.vdim != l.dim || !(l.score_cap >= 0.0)) { why = at + "tied attention sizes"; return LGH_INVALID_ARGUMENT; }
      if (up(l.dim, 64) > kTiedMaxDim) { why = at + "heads above " + std::to_string(kTiedMaxDim); return LGH_UNSUPPORTED; }
    } else if (ga || la) {
      if (ga) {
        if (!l.kv_heads || l.heads % l.kv_heads || l.rot_dims > l.dim || l.rot_dims % 2 || (l.rot_dims && !(l.rot_base > 0.0))) { why = at + "gated attention sizes"; return LGH_INVALID_ARGUMENT; }
        if (l.sink_one > 1 || ((l.sink_one || l.kv_from) && !gr)) { why = at + "a sink or shared keys need grouped attention"; return LGH_UNSUPPORTED; }
        if (l.kv_from) {
          const lgh_layer_desc& o = L[l.kv_from <= i ? l.kv_from - 1 : i];
          if (l.kv_from > i || o.mixer != l.mixer || o.kv_from || o.kv_heads != l.kv_heads || o.heads != l.heads || o.dim != l.dim || o.vdim != l.vdim) {
            why = at + "no such keys and values in layer " + std::to_string(l.kv_from - 1);
            return LGH_INVALID_ARGUMENT;
          }
        }
        if (up(l.dim, 64) > kGattnMaxDim || up(l.vdim, 64) > kGattnMaxDim) { why = at + "heads above " + std::to_string(kGattnMaxDim); return LGH_UNSUPPORTED; }
      }
      if (la && (!l.gla_heads || !l.gla_dim || !l.gla_vdim || !l.gla_rank || !(l.gla_tau > 0.0))) { why = at + "linear attention sizes"; return LGH_INVALID_ARGUMENT; }
      if (!std::isfinite(l.left_scale) || !std::isfinite(l.right_scale)) { why = at + "scales of the two sides"; return LGH_INVALID_ARGUMENT; }
    } else if (l.mixer == LGH_MIXER_DELTA) {
      if (!l.kv_heads || l.heads % l.kv_heads || !l.taps) { why = at + "delta rule sizes"; return LGH_INVALID_ARGUMENT; }
      if (l.taps > kMaxRecTaps) { why = at + "convolution taps"; return LGH_UNSUPPORTED; }
      if (up(l.dim, 16) > 16384 || 2 * l.kv_heads + l.heads > 65535) { why = at + "delta rule heads"; return LGH_UNSUPPORTED; }
    } else if (l.mixer == LGH_MIXER_GLRU) {
      if (l.vdim != l.dim || !l.taps) { why = at + "linear recurrence sizes"; return LGH_INVALID_ARGUMENT; }
      if (l.taps > kMaxRecTaps) { why = at + "convolution taps"; return LGH_UNSUPPORTED; }
    } else if (l.mixer == LGH_MIXER_MLSTM) {
      if (!(l.gate_cap > 0.0)) { why = at + "gate_cap"; return LGH_INVALID_ARGUMENT; }
    } else { why = at + "unknown mixer"; return LGH_UNSUPPORTED; }
  }
  return LGH_OK;
}

// rows of a fused product: segments one below another, each starting at a multiple of 16
static uint32_t seg(LinW& W, uint32_t rows) {
  const uint32_t at = up(W.n, 16);
  W.n = at + rows;
  return at;
}

static void add_mat(LayeredModel& m, const std::string& nm, LinW* W, uint32_t row0, uint32_t n, uint32_t k, int mode = 0) {
  LayeredSlot s;
  s.mat = W; s.row0 = row0; s.n = n; s.k = k; s.mode = mode;
  m.slots[nm] = s;
}
static void add_vec(LayeredModel& m, const std::string& nm, float** v, uint32_t n) {
  LayeredSlot s;
  s.vec = v; s.n = n;
  m.slots[nm] = s;
}
// part of a fused product's bias, at its rows
static void add_bias(LayeredModel& m, const std::string& nm, float** v, uint32_t off, uint32_t n, uint32_t total) {
  add_vec(m, nm, v, n);
  m.slots[nm].off = off;
  m.slots[nm].total = total;
}

// a norm of LGH_RESIDUAL_SANDWICH_DYT: weight, bias and the factor inside
static void add_dyt(LayeredModel& m, const std::string& nm, LayeredNorm& n) {
  add_vec(m, nm, &n.w, m.d.width);
  add_vec(m, nm + ".b", &n.b, m.d.width);
  add_vec(m, nm + ".alpha", &n.alpha, 1);
}
// the norms around a sublayer ("1": mixer, "2": feed-forward)
static void add_sub(LayeredModel& m, const std::string& p, const char* which, float** post_ln, float** post, float** ls) {
  m.n_sub++;
  if (m.ln2()) {
    add_vec(m, p + "norm" + which + "b", post, m.d.width);
    add_vec(m, p + "ls" + which, ls, m.d.width);
  }
  if (!m.dyt()) { add_vec(m, p + "norm" + which, post_ln, m.d.width); return; }
  m.subs.emplace_back();                   // (never grows beyond what was reserved: the slots keep addresses)
  LayeredSub& s = m.subs.back();
  add_dyt(m, p + "norm" + which, s.pre);
  add_dyt(m, p + "norm" + which + "b", s.post);
  if (m.d.conv_taps) add_vec(m, p + "canon" + which, &s.conv, m.d.width * m.d.conv_taps);
}

// sizes, offsets and the tensor table of every layer
static void layered_plan(LayeredModel& m) {
  const lgh_layered_desc& d = m.d;
  const uint32_t W = d.width;
  {
    LayeredSlot s;
    s.raw = &m.embed; s.n = d.vocab_size; s.k = W;
    if (!d.tied_head) m.slots["embed"] = s;
    if (d.bigram_buckets) { s.raw = &m.bigram; s.n = d.bigram_buckets + 1; m.slots["bigram"] = s; }
  }
  auto whole = [&](LinW& L, uint32_t n, uint32_t k) { L.n = n; L.k = k; L.kp = up(k, 64); };
  m.subs.reserve(2 * (size_t)d.num_layers);
  for (uint32_t i = 0; i < d.num_layers; i++) {
    LayeredLayer& L = m.layers[i];
    const lgh_layer_desc& l = L.d;
    const std::string p = "l" + std::to_string(i) + ".";
    add_sub(m, p, "1", &L.norm1, &L.post1, &L.ls1);
    L.in.k = W; L.in.kp = up(W, 64);
    const uint32_t vd = l.mixer == LGH_MIXER_GLA ? 0 : l.heads * l.vdim;
    auto in_seg = [&](const char* nm, uint32_t rows) { const uint32_t at = seg(L.in, rows); add_mat(m, p + "mix." + nm, &L.in, at, rows, W); return at; };
    if (L.latent()) {
      LatentShape& s = L.ls;
      s.heads = l.heads; s.dim = l.dim; s.rot_dim = l.rot_dim; s.rot_n = l.rot_dims; s.vdim = l.vdim; s.rank = l.kv_rank;
      s.ldc = up(l.kv_rank + l.rot_dim, 64);   // (a whole row is also the input row of the expansions)
      s.dimp = up(l.dim, 8);
      s.rankp = up(l.kv_rank, 64);
      s.scale = (float)l.scale; s.eps = (float)d.norm_eps;
      s.window = l.window ? l.window : 0xFFFFFFFFu;
      s.halves = l.rot_form == LGH_ROT_HALVES; s.gate_values = l.gate_form == LGH_GATE_VALUES;
      const uint32_t qrows = l.heads * (l.dim + l.rot_dim);
      s.off_q = in_seg(l.q_rank ? "dq" : "q", l.q_rank ? l.q_rank : qrows);
      s.off_dkv = in_seg("dkv", l.kv_rank + l.rot_dim);
      s.off_g = in_seg("g", s.gate_values ? vd : l.heads);
      L.in.n = up(L.in.n, 16);
      s.ldcat = s.ldq = L.in.n;
      if (l.q_rank) {
        whole(L.uq, qrows, l.q_rank);
        add_mat(m, p + "mix.uq", &L.uq, 0, qrows, l.q_rank);
        add_vec(m, p + "mix.dq.norm", &L.dq_norm, l.q_rank);
        s.ldq = up(qrows, 4);
        m.max_lq = std::max(m.max_lq, s.ldq);
        m.max_qrank = std::max(m.max_qrank, L.uq.kp);
      }
      add_vec(m, p + "mix.dkv.norm", &L.dkv_norm, l.kv_rank);
      whole(L.uk, l.heads * l.dim, l.kv_rank);
      whole(L.uv, vd, l.kv_rank);
      add_mat(m, p + "mix.uk", &L.uk, 0, L.uk.n, l.kv_rank);
      m.slots[p + "mix.uk"].transpose = &L;
      add_mat(m, p + "mix.uv", &L.uv, 0, vd, l.kv_rank);
    } else if (L.tied()) {
      TiedShape& s = L.ts;
      s.heads = l.heads; s.kv_heads = l.kv_heads; s.dim = l.dim; s.dp = up(l.dim, 64);
      s.window = l.window ? l.window : 0xFFFFFFFFu; s.keep = l.keep_first;
      s.rows = up(d.max_seq_len, 64);
      s.scale = (float)l.scale; s.cap = (float)l.score_cap; s.eps = (float)d.norm_eps;
      s.off_q = in_seg("q", vd);
      s.off_k = in_seg("k", l.kv_heads * l.dim);
      L.in.n = up(L.in.n, 16);
      s.ldcat = L.in.n;
      add_vec(m, p + "mix.q.norm", &L.qn, vd);
      add_vec(m, p + "mix.k.norm", &L.kn, l.kv_heads * l.dim);
      add_vec(m, p + "mix.temp", &L.temp, l.heads);
      add_vec(m, p + "mix.sink", &L.sink, l.heads);
      L.splits = tied_splits(s, d.max_seq_len, 1, m.f32, m.forced_splits);
      for (uint32_t t = 1; t <= kTiedShort; t++) {
        const size_t rows = (size_t)t * l.heads * tied_splits(s, d.max_seq_len, t, m.f32, m.forced_splits);
        m.max_tied_rows = std::max(m.max_tied_rows, rows);
        m.max_tied_acc = std::max(m.max_tied_acc, rows * l.dim);
      }
      m.max_tied_q = std::max(m.max_tied_q, l.heads * s.dp);
    } else if (L.delta()) {
      DeltaShape& s = L.des;
      s.heads = l.heads; s.kv_heads = l.kv_heads; s.dim = l.dim; s.vdim = l.vdim; s.taps = l.taps; s.dk = up(l.dim, 16); s.lv = up(l.vdim, 16);
      s.eps = (float)d.norm_eps;
      const uint32_t qk = l.kv_heads * l.dim;
      s.off_q = in_seg("q", qk);
      s.off_k = in_seg("k", qk);
      s.off_v = in_seg("v", vd);
      s.cols = s.off_v + vd;
      s.off_g = in_seg("g", vd);
      s.off_b = in_seg("b", l.heads);
      s.off_a = in_seg("a", l.heads);
      L.in.n = up(L.in.n, 16);
      s.ldcat = L.in.n;
      add_bias(m, p + "mix.q.conv", &L.conv, s.off_q * l.taps, qk * l.taps, s.cols * l.taps);
      add_bias(m, p + "mix.k.conv", &L.conv, s.off_k * l.taps, qk * l.taps, s.cols * l.taps);
      add_bias(m, p + "mix.v.conv", &L.conv, s.off_v * l.taps, vd * l.taps, s.cols * l.taps);
      add_vec(m, p + "mix.A_log", &L.a_log, l.heads);
      add_vec(m, p + "mix.dt_bias", &L.dt, l.heads);
      add_vec(m, p + "mix.norm", &L.gnorm, l.vdim);
      m.recurrent = true;
      m.max_num = std::max(m.max_num, l.heads * s.lv);
      m.max_dqk = std::max(m.max_dqk, l.kv_heads * s.dk);
      m.max_dw = std::max(m.max_dw, l.heads * s.dk);
      m.max_dv = std::max(m.max_dv, l.heads * s.lv);
      m.max_dheads = std::max(m.max_dheads, l.heads);
    } else if (L.glru()) {
      GlruShape& s = L.rs;
      s.width = vd; s.blocks = l.heads; s.bs = l.dim; s.taps = l.taps;
      s.off_y = in_seg("y", vd);
      s.off_x = in_seg("x", vd);
      L.in.n = up(L.in.n, 16);
      s.ldcat = L.in.n;
      add_bias(m, p + "mix.y.b", &L.in_bias, s.off_y, vd, L.in.n);
      add_bias(m, p + "mix.x.b", &L.in_bias, s.off_x, vd, L.in.n);
      add_vec(m, p + "mix.conv", &L.conv, vd * l.taps);
      add_vec(m, p + "mix.conv.b", &L.conv_b, vd);
      s.gate_rows = 2 * up(l.dim, 16);
      whole(L.gates, l.heads * s.gate_rows, l.dim);
      s.gate_kp = L.gates.kp;
      for (int i = 0; i < 2; i++) {
        const std::string nm = p + (i ? "mix.ri" : "mix.ra");
        add_mat(m, nm, &L.gates, 0, vd, l.dim, 1 + i);
        m.slots[nm].parts = l.heads;
        m.slots[nm].stride = s.gate_rows;
        add_vec(m, nm + ".b", i ? &L.ib : &L.rb, vd);
      }
      add_vec(m, p + "mix.lam", &L.lam, vd);
      m.recurrent = true;
      m.max_rec = std::max(m.max_rec, vd);
    } else if (L.gattn() || L.gla()) {
      const bool par = l.mixer == LGH_MIXER_PARALLEL;
      const std::string left = par ? "left." : "", right = par ? "right." : "", pl = p + "mix." + left, pr = p + "mix." + right;
      if (L.gattn()) {
        GattnShape& s = L.gs;
        s.heads = l.heads; s.kv_heads = l.kv_heads; s.dim = l.dim; s.vdim = l.vdim; s.dp = up(l.dim, 64); s.vp = up(l.vdim, 64);
        s.chunk = l.chunk ? l.chunk : 0xFFFFFFFFu; s.window = L.grouped() && l.window ? l.window : 0xFFFFFFFFu; s.rot_n = l.rot_dims;
        s.gated = !L.grouped(); s.sink = l.sink_one;
        s.rows = up(d.max_seq_len, 64);
        s.scale = (float)l.scale; s.eps = (float)d.norm_eps; s.out_scale = par ? (float)l.left_scale : 1.0f;
        s.off_q = in_seg((left + "q").c_str(), l.heads * l.dim);
        if (!l.kv_from) {
          s.off_k = in_seg((left + "k").c_str(), l.kv_heads * l.dim);
          s.off_v = in_seg((left + "v").c_str(), l.kv_heads * l.vdim);
        }
        if (s.gated) {
          s.off_g = in_seg((left + "g").c_str(), vd);
          add_vec(m, pl + "q.norm", &L.qn, l.dim);
          add_vec(m, pl + "k.norm", &L.kn, l.dim);
        } else {
          add_vec(m, pl + "o.b", &L.out_bias, W);
        }
        L.splits = gattn_splits(s, d.max_seq_len, 1, m.f32, m.forced_splits);
        for (uint32_t t = 1; t <= kGattnShort; t++) {
          const size_t rows = (size_t)t * l.heads * gattn_splits(s, d.max_seq_len, t, m.f32, m.forced_splits);
          m.max_tied_rows = std::max(m.max_tied_rows, rows);
          m.max_tied_acc = std::max(m.max_tied_acc, rows * l.vdim);
        }
        if (s.dp <= kGattnFlashDim) m.max_tied_q = std::max(m.max_tied_q, l.heads * s.dp);
      }
      if (L.gla()) {
        GlaShape& s = L.as;
        s.heads = l.gla_heads; s.dim = l.gla_dim; s.vdim = l.gla_vdim; s.rank = l.gla_rank;
        s.lds = up(s.vdim, 16); s.ldo = up(s.vdim, 4);
        s.tau = (float)l.gla_tau; s.eps = (float)d.norm_eps; s.out_scale = par ? (float)l.right_scale : 1.0f;
        s.off_q = in_seg((right + "q").c_str(), s.heads * s.dim);
        s.off_k = in_seg((right + "k").c_str(), s.heads * s.dim);
        s.off_v = in_seg((right + "v").c_str(), s.heads * s.vdim);
        s.off_g = in_seg((right + "g").c_str(), s.heads * s.vdim);
        s.off_a = in_seg((right + "a1").c_str(), s.rank);
        whole(L.a2, s.heads * s.dim, s.rank);
        s.a2_ld = L.a2.kp;
        add_mat(m, pr + "a2", &L.a2, 0, L.a2.n, s.rank);
        add_vec(m, pr + "a2.b", &L.a2b, L.a2.n);
        add_vec(m, pr + "norm", &L.gnorm, s.vdim);
        m.recurrent = true;
        m.max_num = std::max(m.max_num, s.heads * s.ldo);
        m.max_gla = std::max(m.max_gla, s.heads * s.dim);
      }
      L.in.n = up(L.in.n, 16);
      L.gs.ldcat = L.as.ldcat = L.in.n;
      if (L.gattn()) {
        add_bias(m, pl + "q.b", &L.in_bias, L.gs.off_q, l.heads * l.dim, L.in.n);
        if (!l.kv_from) {
          add_bias(m, pl + "k.b", &L.in_bias, L.gs.off_k, l.kv_heads * l.dim, L.in.n);
          add_bias(m, pl + "v.b", &L.in_bias, L.gs.off_v, l.kv_heads * l.vdim, L.in.n);
        }
      }
      // both sides' output projections side by side: one product
      L.gla_col = up(vd, 64);
      const uint32_t cols = L.gla() ? L.gla_col + L.as.heads * L.as.vdim : vd;
      whole(L.out, W, cols);
      if (L.gattn()) add_mat(m, pl + "o", &L.out, 0, W, vd);
      if (L.gla()) {
        add_mat(m, pr + "o", &L.out, 0, W, L.as.heads * L.as.vdim);
        m.slots[pr + "o"].col0 = L.gla_col;
      }
    } else {
      MlstmShape& s = L.ms;
      s.heads = l.heads; s.dim = l.dim; s.vdim = l.vdim;
      s.lds = up(l.vdim + 1, 16); s.ldo = up(l.vdim + 2, 4);
      s.cap = (float)l.gate_cap; s.eps = (float)d.norm_eps;
      s.off_q = in_seg("q", l.heads * l.dim);
      s.off_k = in_seg("k", l.heads * l.dim);
      s.off_v = in_seg("v", vd);
      s.off_g = in_seg("g", vd);
      s.off_i = in_seg("i", l.heads);
      s.off_f = in_seg("f", l.heads);
      L.in.n = up(L.in.n, 16);
      s.ldcat = s.ldqk = L.in.n;
      add_vec(m, p + "mix.i.b", &L.bi, l.heads);
      add_vec(m, p + "mix.f.b", &L.bf, l.heads);
      add_vec(m, p + "mix.norm", &L.mnorm, vd);
      m.recurrent = true;
      m.max_num = std::max(m.max_num, l.heads * s.ldo);
    }
    m.max_cat = std::max(m.max_cat, L.in.n);
    if (!L.out.n) {
      whole(L.out, W, vd);
      add_mat(m, p + "mix.o", &L.out, 0, W, vd);
    }
    m.max_ao = std::max(m.max_ao, L.out.kp);
    if (L.moe()) {
      add_sub(m, p, "2", &L.norm2, &L.post2, &L.ls2);
      whole(L.router, l.experts + l.identity, W);
      add_mat(m, p + "mlp.router", &L.router, 0, L.router.n, W);
      if (l.router_form == LGH_ROUTER_SOFTMAX_GROUPS) add_vec(m, p + "mlp.correction", &L.correction, L.router.n);
      L.egu_rows = 2 * up(l.ff, 16);
      L.edown_rows = up(W, 16);
      whole(L.egu, l.experts * L.egu_rows, W);
      L.egu.paired = true;
      whole(L.edown, l.experts * L.edown_rows, l.ff);
      for (uint32_t e = 0; e < l.experts; e++) {
        const std::string pe = p + "mlp.e" + std::to_string(e) + ".";
        add_mat(m, pe + "gate", &L.egu, e * L.egu_rows, l.ff, W, 1);
        add_mat(m, pe + "up", &L.egu, e * L.egu_rows, l.ff, W, 2);
        add_mat(m, pe + "down", &L.edown, e * L.edown_rows, W, l.ff);
      }
      if (l.shared_ff) {
        whole(L.gu, 2 * up(l.shared_ff, 16), W);
        L.gu.paired = true;
        add_mat(m, p + "mlp.shared.gate", &L.gu, 0, l.shared_ff, W, 1);
        add_mat(m, p + "mlp.shared.up", &L.gu, 0, l.shared_ff, W, 2);
        whole(L.down, W, l.shared_ff);
        add_mat(m, p + "mlp.shared.down", &L.down, 0, W, l.shared_ff);
      }
      m.max_act = std::max(m.max_act, L.act_cols());
      m.max_experts = std::max(m.max_experts, l.experts + l.identity);
      m.max_top = std::max(m.max_top, l.top);
      m.max_pair_act = std::max(m.max_pair_act, l.top * L.edown.kp);
    } else if (l.ff_kind) {
      add_sub(m, p, "2", &L.norm2, &L.post2, &L.ls2);
      if (l.ff_kind == LGH_FF_RELU2) {
        whole(L.gu, l.ff, W);
        add_mat(m, p + "mlp.up", &L.gu, 0, l.ff, W);
      } else {
        whole(L.gu, 2 * up(l.ff, 16), W);
        L.gu.paired = true;
        add_mat(m, p + "mlp.gate", &L.gu, 0, l.ff, W, 1);
        add_mat(m, p + "mlp.up", &L.gu, 0, l.ff, W, 2);
      }
      whole(L.down, W, l.ff);
      add_mat(m, p + "mlp.down", &L.down, 0, W, l.ff);
      m.max_act = std::max(m.max_act, L.down.kp);
    }
  }
  if (m.dyt()) add_dyt(m, "final.norm", m.final_dyt);
  else add_vec(m, "final.norm", &m.final_norm, W);
  whole(m.head, d.vocab_size, W);
  add_mat(m, d.tied_head ? "embed" : "head", &m.head, 0, d.vocab_size, W);
}

extern "C" int lgh_create_layered(const lgh_layered_desc* desc, const lgh_layer_desc* layers, lgh_ctx** out) {
  if (!desc || !layers || !out || desc->struct_size != sizeof(lgh_layered_desc)) return LGH_INVALID_ARGUMENT;
  *out = nullptr;
  if (desc->flags & LGH_FLAG_REMOVED_MASK) return LGH_UNSUPPORTED;
  std::string why;
  if (int rc = layered_check(*desc, layers, why)) return rc;
  const int ndev = lgh_device_count();
  if (ndev <= 0 || desc->device_id < 0 || desc->device_id >= ndev) return LGH_NOT_AVAILABLE;
  lgh_ctx* c = new lgh_ctx();
  lgh_model_desc& d = c->d;   // what the engine's shared entry points read
  d.struct_size = sizeof(d);
  d.hidden_size = desc->width; d.vocab_size = desc->vocab_size; d.num_layers = desc->num_layers; d.max_seq_len = desc->max_seq_len;
  d.norm_eps = (float)desc->norm_eps; d.device_id = desc->device_id; d.flags = desc->flags & ~(uint32_t)LGH_FLAG_KV_INT8;
  c->device = d.device_id;
  c->l0 = 0; c->l1 = d.num_layers;
  c->direct_attn_max_kv = 0;   // one attention structure
  if (hipSetDevice(c->device) != hipSuccess || hipStreamCreateWithFlags(&c->own_stream, hipStreamNonBlocking) != hipSuccess) {
    delete c;
    return LGH_INITIALIZATION_FAILED;
  }
  c->stream = c->own_stream;
  LayeredModel* m = new LayeredModel();
  c->lm = m;
  m->d = *desc;
  m->f32 = desc->compute == LGH_COMPUTE_F32;
  m->forced_splits = (desc->flags >> LGH_FLAG_ATTN_SPLITS_SHIFT) & 0xFFu;
  m->layers.resize(d.num_layers);
  for (uint32_t i = 0; i < d.num_layers; i++) m->layers[i].d = layers[i];
  layered_plan(*m);
  *out = c;
  return LGH_OK;
}

static int zeroed(lgh_ctx* c, void** p, size_t bytes, uint64_t* account) {
  if (int rc = dev_alloc(c, p, bytes)) return rc;
  if (bytes) L_TRY(c, LGH_OPERATION_FAILED, hipMemsetAsync(*p, 0, bytes, c->stream));
  if (account) *account += bytes;
  return LGH_OK;
}

int layered_upload(lgh_ctx* c, const char* name, uint32_t type, const uint64_t ne[4], const void* host, size_t nbytes) {
  LayeredModel& m = *c->lm;
  const std::string nm(name);
  auto it = m.slots.find(nm);
  if (it == m.slots.end()) return fail(c, LGH_INVALID_ARGUMENT, "unknown tensor name " + nm);
  LayeredSlot& s = it->second;
  const uint64_t n0 = ne[0], n1 = ne[1] ? ne[1] : 1, n2 = ne[2] ? ne[2] : 1;
  int rc;
  if (s.vec) {
    if (n0 * n1 * n2 != s.n) return fail(c, LGH_SHAPE_MISMATCH, nm + ": expected " + std::to_string(s.n) + " elements");
    if (s.total) {                           // a part of a vector that several tensors share
      if (!*s.vec && (rc = zeroed(c, (void**)s.vec, (size_t)s.total * 4, nullptr))) return rc;
      L_TRY(c, LGH_OPERATION_FAILED, hipStreamSynchronize(c->stream));
      float* at = *s.vec + s.off;
      if ((rc = upload_f32(c, &at, (int)type, s.n, host, nbytes))) return rc;
      c->stats.weight_bytes += s.done ? 0 : (uint64_t)s.n * 4;
    } else if ((rc = upload_f32(c, s.vec, (int)type, s.n, host, nbytes))) return rc;
    s.done = true;
    return LGH_OK;
  }
  if (type != LGH_TYPE_BF16) return fail(c, LGH_DTYPE_MISMATCH, nm + ": matrices of this model are bf16");
  if (n0 != s.k || n1 != s.n / s.parts || n2 != s.parts) return fail(c, LGH_SHAPE_MISMATCH, nm + ": expected [" + std::to_string(s.k) + "," + std::to_string(s.n) + "]");
  if (nbytes != (size_t)s.n * s.k * 2) return fail(c, LGH_SHAPE_MISMATCH, nm + ": byte size does not match its shape");
  if (s.raw) {
    if (!*s.raw && (rc = dev_alloc(c, (void**)s.raw, nbytes))) return rc;
    L_TRY(c, LGH_OPERATION_FAILED, hipMemcpy(*s.raw, host, nbytes, hipMemcpyHostToDevice));
    c->stats.weight_bytes += s.done ? 0 : nbytes;
    s.done = true;
    return LGH_OK;
  }
  LinW& W = *s.mat;
  if (!W.w && (rc = zeroed(c, (void**)&W.w, (size_t)W.np() * W.kp * 2, nullptr))) return rc;
  void* raw = nullptr;
  L_TRY(c, LGH_ALLOCATION_FAILED, hipMalloc(&raw, nbytes));
  hipError_t e = hipMemcpy(raw, host, nbytes, hipMemcpyHostToDevice);
  for (uint32_t i = 0; i < s.parts && e == hipSuccess; i++)
    e = lin_pack_launch((const uint16_t*)raw + (size_t)i * (s.n / s.parts) * s.k, s.n / s.parts, s.k, W.w + s.col0, W.kp, s.row0 + i * s.stride, s.mode, c->stream);
  if (e == hipSuccess && s.transpose) {
    LayeredLayer& L = *s.transpose;
    const size_t tb = (size_t)L.ls.heads * L.ls.rank * L.ls.dimp * 2;
    if (!L.uk_t && (rc = zeroed(c, (void**)&L.uk_t, tb, nullptr))) { (void)hipFree(raw); return rc; }
    e = lin_transpose_heads_launch((const uint16_t*)raw, L.ls.heads, L.ls.dim, L.ls.rank, L.uk_t, L.ls.dimp, c->stream);
  }
  if (e == hipSuccess) e = hipStreamSynchronize(c->stream);
  (void)hipFree(raw);
  if (e != hipSuccess) return fail(c, LGH_OPERATION_FAILED, nm + ": " + hipGetErrorString(e));
  c->stats.weight_bytes += s.done ? 0 : nbytes;
  s.done = true;
  return LGH_OK;
}

// cos / sin of every position: angles in 64-bit, with the YaRN blend of frequencies when the layer asks for it
static std::vector<float> rotation_table(const lgh_layer_desc& l, uint32_t max_seq) {
  const uint32_t np = l.rot_dims / 2;
  std::vector<double> f(np);
  for (uint32_t i = 0; i < np; i++) f[i] = std::pow(l.rot_base, -2.0 * i / l.rot_dims);
  double mag = 1.0;
  if (l.yarn_factor > 0.0) {
    auto turn = [&](double t) { return l.rot_dims * std::log(l.yarn_original / (2.0 * M_PI * t)) / (2.0 * std::log(l.rot_base)); };
    const double lo = std::max(std::floor(turn(l.yarn_fast)), 0.0), hi = std::min(std::ceil(turn(l.yarn_slow)), (double)l.rot_dims - 1.0);
    for (uint32_t i = 0; i < np; i++) {
      const double ramp = std::min(std::max((i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
      f[i] = f[i] / l.yarn_factor * ramp + f[i] * (1.0 - ramp);
    }
    mag = 0.1 * std::log(l.yarn_factor) + 1.0;
  }
  std::vector<float> cs((size_t)max_seq * np * 2);
  for (uint32_t p = 0; p < max_seq; p++)
    for (uint32_t i = 0; i < np; i++) {
      cs[((size_t)p * np + i) * 2] = (float)(std::cos(p * f[i]) * mag);
      cs[((size_t)p * np + i) * 2 + 1] = (float)(std::sin(p * f[i]) * mag);
    }
  return cs;
}

int layered_finalize(lgh_ctx* c) {
  LayeredModel& m = *c->lm;
  std::string missing;
  for (auto& s : m.slots)
    if (!s.second.done) missing += (missing.empty() ? "" : ", ") + s.first;
  if (!missing.empty()) return fail(c, LGH_INITIALIZATION_FAILED, "missing tensors: " + missing.substr(0, 400));
  const lgh_layered_desc& d = m.d;
  int rc;
  uint32_t max_rows = 0, max_rank = 0, max_ldc = 0;
  for (uint32_t i = 0; i < d.num_layers; i++) {
    LayeredLayer& L = m.layers[i];
    if (L.rotated()) {
      for (uint32_t j = 0; j < i && !L.cs; j++) {   // layers with the same rotation share its table
        const lgh_layer_desc &a = L.d, &b = m.layers[j].d;
        if (m.layers[j].rotated() && a.rot_dims == b.rot_dims && a.rot_base == b.rot_base && a.yarn_factor == b.yarn_factor &&
            a.yarn_original == b.yarn_original && a.yarn_fast == b.yarn_fast && a.yarn_slow == b.yarn_slow)
          L.cs = m.layers[j].cs;
      }
      if (!L.cs) {
        const std::vector<float> cs = rotation_table(L.d, d.max_seq_len);
        if ((rc = zeroed(c, (void**)&L.cs, cs.size() * 4, &c->stats.scratch_bytes))) return rc;
        L_TRY(c, LGH_OPERATION_FAILED, hipStreamSynchronize(c->stream));
        if (!cs.empty()) L_TRY(c, LGH_OPERATION_FAILED, hipMemcpy(L.cs, cs.data(), cs.size() * 4, hipMemcpyHostToDevice));
      }
    }
    if (L.d.kv_from) {                     // an earlier layer's cache rows
      L.cache = m.layers[L.d.kv_from - 1].cache;
      L.vcache = m.layers[L.d.kv_from - 1].vcache;
    } else if (L.delta()) {
      if ((rc = zeroed(c, (void**)&L.S, (size_t)L.des.heads * L.des.dk * L.des.lv * 4, &c->stats.kv_bytes))) return rc;
      if ((rc = zeroed(c, (void**)&L.rhist, (size_t)L.des.taps * L.des.cols * 4, &c->stats.kv_bytes))) return rc;
    } else if (L.latent()) {
      if ((rc = zeroed(c, &L.cache, (size_t)d.max_seq_len * L.ls.ldc * m.el(), &c->stats.kv_bytes))) return rc;
      max_rows = std::max(max_rows, L.ls.heads); max_rank = std::max(max_rank, L.ls.rank); max_ldc = std::max(max_ldc, L.ls.ldc);
    } else if (L.tied()) {
      if ((rc = zeroed(c, &L.cache, (size_t)L.ts.kv_heads * L.ts.rows * L.ts.dp * m.el(), &c->stats.kv_bytes))) return rc;
      if ((rc = zeroed(c, (void**)&L.kinv, (size_t)L.ts.rows * 4, &c->stats.kv_bytes))) return rc;
    } else if (L.glru()) {
      if ((rc = zeroed(c, (void**)&L.rS, (size_t)L.rs.width * 4, &c->stats.kv_bytes))) return rc;
      if ((rc = zeroed(c, (void**)&L.rhist, (size_t)L.rs.taps * L.rs.width * 4, &c->stats.kv_bytes))) return rc;
    } else if (L.gattn() || L.gla()) {
      if (L.gattn()) {
        if ((rc = zeroed(c, &L.cache, (size_t)L.gs.kv_heads * L.gs.rows * L.gs.dp * m.el(), &c->stats.kv_bytes))) return rc;
        if ((rc = zeroed(c, &L.vcache, (size_t)L.gs.kv_heads * L.gs.rows * L.gs.vp * m.el(), &c->stats.kv_bytes))) return rc;
      }
      if (L.gla() && (rc = zeroed(c, (void**)&L.S, (size_t)L.as.heads * L.as.dim * L.as.lds * 4, &c->stats.kv_bytes))) return rc;
    } else {
      if ((rc = zeroed(c, (void**)&L.S, (size_t)L.ms.heads * L.ms.dim * L.ms.lds * 4, &c->stats.kv_bytes))) return rc;
      if ((rc = zeroed(c, (void**)&L.m, (size_t)2 * L.ms.heads * 8, &c->stats.kv_bytes))) return rc;
    }
  }
  uint32_t splits = m.forced_splits;
  // enough splits that a long context's workgroups cover the chip; no more, since every split's partial sums are merged
  if (!splits) splits = std::min(512 / std::max(1u, (max_rows + 15) / 16), std::min(std::max(d.max_seq_len / 128, 64u), kLatMaxSplits));
  m.n_splits = std::max(1u, std::min(splits, kLatMaxSplits));
  // the absorbed path's rows: one token's heads in decode, several tokens' in short portions
  const size_t rows = max_rows ? kLatAbsorbRows : 0;
  uint64_t* sb = &c->stats.scratch_bytes;
  struct { void** p; size_t n; } bufs[] = {
      {(void**)&m.x[0], (size_t)d.width * 4}, {(void**)&m.x[1], (size_t)d.width * 4}, {(void**)&m.y, (size_t)up(d.width, 16) * 4},
      {(void**)&m.cat, (size_t)m.max_cat * 4}, {(void**)&m.ao, (size_t)m.max_ao * 4}, {(void**)&m.act, (size_t)m.max_act * 4},
      {(void**)&m.num, (size_t)m.max_num * 4}, {(void**)&m.qa, rows * max_ldc * m.el()}, {(void**)&m.lq, (size_t)m.max_lq * 4},
      {(void**)&m.part_ml, std::max(rows * m.n_splits, m.max_tied_rows) * 2 * 4}, {(void**)&m.part_acc, std::max(rows * m.n_splits * max_rank, m.max_tied_acc) * 4},
      {(void**)&m.selw, (size_t)m.max_top * 4},
      {(void**)&m.tokens, (size_t)d.max_seq_len * 4}, {(void**)&m.h, m.dyt() || m.pre() ? (size_t)up(d.width, 16) * 4 : 0}, {(void**)&m.hist, m.hist_floats() * 4},
      {(void**)&m.rlogits, (size_t)m.max_experts * 4}, {(void**)&m.sel, (size_t)m.max_top * 4}, {(void**)&c->logits, (size_t)d.vocab_size * 4}, {(void**)&c->state, ST_WORDS * 4},
      {(void**)&c->amax_v, 64 * 4}, {(void**)&c->amax_i, 64 * 4}, {(void**)&c->tok_log, (size_t)d.max_seq_len * 4},
  };
  for (auto& b : bufs)
    if ((rc = zeroed(c, b.p, b.n, sb))) return rc;
  if (m.ln2())                             // a sublayer's scale per channel goes into the weight of the norm in front of it
    for (LayeredLayer& L : m.layers) {
      L_TRY(c, LGH_OPERATION_FAILED, vec_mul_launch(L.post1, L.ls1, d.width, c->stream));
      if (L.d.ff_kind) L_TRY(c, LGH_OPERATION_FAILED, vec_mul_launch(L.post2, L.ls2, d.width, c->stream));
    }
  // where the residual stream ends up: every sublayer's update swaps the two vectors; channel by channel it stays in place
  c->hidden = m.dyt() ? m.x[0] : m.x[m.n_sub & 1];
  L_TRY(c, LGH_OPERATION_FAILED, hipStreamSynchronize(c->stream));
  return LGH_OK;
}

static EmbedArgs embed_args(const LayeredModel& m) {
  EmbedArgs a{};
  a.embed = m.d.tied_head ? m.head.w : m.embed; a.ld = m.d.tied_head ? m.head.kp : m.d.width; a.bigram = m.bigram; a.width = m.d.width; a.buckets = m.d.bigram_buckets;
  a.mul_prev = m.d.bigram_mul_prev; a.mul_cur = m.d.bigram_mul_cur; a.hist = m.tokens;
  return a;
}

// q: the queries where they are made from their latent
static LatentBufs latent_bufs(const LayeredModel& m, const LayeredLayer& L, const float* cat, const float* q) {
  LatentBufs b{};
  b.cat = cat; b.q = L.d.q_rank ? q : cat + L.ls.off_q; b.dkv_norm = L.dkv_norm; b.cs = L.cs; b.uk_t = L.uk_t; b.uv = L.uv.w; b.cache = L.cache; b.qa = m.qa;
  b.part_ml = m.part_ml; b.part_acc = m.part_acc;
  return b;
}
// shares of the visible keys: no more than a window has tiles
static uint32_t latent_splits(const LayeredModel& m, const LayeredLayer& L) { return std::min(m.n_splits, L.ls.window / 32 + 2); }
static DeltaBufs delta_bufs(const LayeredModel& m, const LayeredLayer& L, const float* cat, float* num) {
  DeltaBufs b{};
  b.cat = cat; b.conv = L.conv; b.a_log = L.a_log; b.dt = L.dt; b.norm = L.gnorm; b.S = L.S; b.hist = L.rhist; b.num = num;
  b.q = m.bdq; b.k = m.bdk; b.v = m.bdv; b.u = m.bdu; b.w = m.bdw; b.p = m.bdp; b.wge = m.bdwge; b.cd = m.bdcd; b.Mcap = up(m.blk, 64);
  return b;
}
static MlstmBufs mlstm_bufs(const LayeredModel& m, const LayeredLayer& L, const float* cat, float* num) {
  MlstmBufs b{};
  b.cat = cat; b.bi = L.bi; b.bf = L.bf; b.norm = L.mnorm; b.S = L.S; b.m = L.m; b.num = num;
  b.u = m.bu; b.mx = m.bmx; b.dec = m.bdec; b.wgt = m.bwgt; b.cdec = m.bcdec; b.a = m.ba; b.nk = m.bnk; b.Mcap = up(m.blk, 64);
  b.qk = cat;
  return b;
}
static GattnBufs gattn_bufs(const LayeredModel& m, const LayeredLayer& L, const float* cat) {
  GattnBufs b{};
  b.cat = cat; b.qn = L.qn; b.kn = L.kn; b.cs = L.cs; b.kc = L.cache; b.vc = L.vcache; b.shared = L.d.kv_from != 0;
  b.part_ml = m.part_ml; b.part_acc = m.part_acc;
  return b;
}
static GlaBufs gla_bufs(const LayeredModel& m, const LayeredLayer& L, const float* cat, float* num) {
  GlaBufs b{};
  b.cat = cat; b.a2 = L.a2.w; b.a2b = L.a2b; b.norm = L.gnorm; b.S = L.S; b.num = num;
  b.qk = m.bqk; b.dec = m.bgdec; b.a = m.ba; b.Mcap = up(m.blk, 64);
  return b;
}
static GlruBufs glru_bufs(const LayeredModel& m, const LayeredLayer& L, const float* cat) {
  GlruBufs b{};
  b.cat = cat; b.conv = L.conv; b.conv_b = L.conv_b; b.gates = L.gates.w; b.rb = L.rb; b.ib = L.ib; b.lam = L.lam; b.S = L.rS; b.hist = L.rhist;
  b.a = m.brec; b.x = m.brec ? m.brec + (size_t)m.blk * m.max_rec : nullptr; b.sum = m.brsum; b.s0 = m.brsum ? m.brsum + (size_t)((m.blk + 63) / 64) * m.max_rec * 2 : nullptr;
  return b;
}

static TiedBufs tied_bufs(const LayeredModel& m, const LayeredLayer& L, const float* cat) {
  TiedBufs b{};
  b.cat = cat; b.qn = L.qn; b.kn = L.kn; b.temp = L.temp; b.sink = L.sink; b.cache = L.cache; b.kinv = L.kinv;
  b.part_ml = m.part_ml; b.part_acc = m.part_acc;
  return b;
}
static DytW dyt_w(const LayeredNorm& n) {
  DytW r;
  r.w = n.w; r.b = n.b; r.alpha = n.alpha;
  return r;
}
// the convolution in front of sublayer i
static ConvW conv_w(const LayeredModel& m, uint32_t i) {
  ConvW r;
  if (!m.d.conv_taps) return r;
  r.w = m.subs[i].conv; r.taps = m.d.conv_taps;
  r.hist = m.d.conv_taps > 1 ? m.hist + (size_t)i * (m.d.conv_taps - 1) * m.d.width : nullptr;
  return r;
}
// decode: what the product that ends sublayer i does to the stream, up to the input of sublayer i + 1 (the last one: of the output projection)
static PostUpdate post_update(const lgh_ctx* c, int i) {
  const LayeredModel& m = *c->lm;
  PostUpdate p;
  p.x = m.x[0]; p.xout = m.x[0]; p.hout = m.h; p.pos = c->state + ST_POS; p.mult = (float)m.d.residual_mult; p.width = m.d.width;
  if (i >= 0) p.post = dyt_w(m.subs[i].post);
  if (i + 1 < (int)m.n_sub) { p.next = dyt_w(m.subs[i + 1].pre); p.conv = conv_w(m, i + 1); }
  else p.next = dyt_w(m.final_dyt);
  return p;
}

// bytes of one token's attention / recurrence in a layer at the current position
static uint64_t mixer_bytes(const lgh_ctx* c, const LayeredLayer& L) {
  if (L.tied()) {
    const uint64_t p = c->pos + 1, w = std::min<uint64_t>(p, L.ts.window), n = w + std::min<uint64_t>(L.ts.keep, p - w);
    return n * ((uint64_t)L.ts.kv_heads * L.ts.dim * c->lm->el() + 4);
  }
  if (L.glru()) return L.gates.bytes() + (uint64_t)L.rs.width * (L.rs.taps * 2 + 7) * 4;
  if (L.gattn() || L.gla()) {
    uint64_t b = 0;
    if (L.gattn()) b += std::min<uint64_t>(c->pos + 1 - c->pos / L.gs.chunk * L.gs.chunk, L.gs.window) * L.gs.kv_heads * (L.gs.dim + L.gs.vdim) * c->lm->el();
    if (L.gla()) b += (uint64_t)L.as.heads * L.as.dim * L.as.vdim * 8 + L.a2.bytes();
    return b;
  }
  if (L.delta()) return (uint64_t)L.des.heads * L.des.dim * L.des.vdim * 8 + (uint64_t)L.des.cols * (L.des.taps * 2 + 1) * 4;
  if (L.latent()) return std::min<uint64_t>(c->pos + 1, L.ls.window) * (L.ls.rank + L.ls.rot_dim) * c->lm->el();
  return (uint64_t)L.ms.heads * L.ms.dim * (L.ms.vdim + 1) * 8;   // state read and written
}

int layered_enqueue_token(lgh_ctx* c, int mode) {
  LayeredModel& m = *c->lm;
  hipStream_t st = c->stream;
  const int* pos = c->state + ST_POS;
  int rc;
  if ((rc = run_k(c, LGH_K_EMBED, LGH_SYM_EMBED, (uint64_t)m.d.width * 4, [&] {
         const PostUpdate first = m.dyt() ? post_update(c, -1) : PostUpdate();
         return layered_embed_launch(embed_args(m), c->state, m.x[0], m.dyt() ? &first : nullptr, st);
       })))
    return rc;
  uint32_t cur = 0;
  int sub = 0;
  const float* pend = nullptr;   // norm weight of the sublayer output waiting in m.y (LGH_RESIDUAL_PRE_RMS: any)
  auto mv = [&](int cls, const LinW& W, float* out, LinMv a, int pro) {
    a.w = W.w; a.n = W.n; a.kp = W.kp; a.k = W.k; a.paired = W.paired; a.out = out;
    return run_k(c, cls, LGH_SYM_LINEAR, W.bytes(), [&] { return lin_mv_launch(pro, a, st); });
  };
  auto mv_end = [&](int cls, const LinW& W, LinMv a, int pro, float* norm) {   // the product that ends a sublayer
    if (m.dyt()) a.post = post_update(c, sub++);
    else pend = norm;
    return mv(cls, W, m.y, a, pro);
  };
  // a product's input: the residual stream, or what was made of it.  pre: the sublayer's norm in front (LGH_RESIDUAL_PRE_RMS); nw2: the final norm
  auto read = [&](LinMv& a, const float* pre, const float* nw2 = nullptr) -> int {
    a.x = m.dyt() ? m.h : m.x[cur];
    int pro = LP_COPY;
    if (m.ln2()) {
      a.nw2 = nw2 ? nw2 : pre; a.eps = (float)m.d.norm_eps; a.mult = (float)m.d.residual_mult;
      if (pend) {
        a.y = m.y; a.nw = pend; a.xout = m.x[cur ^ 1];
        cur ^= 1;
        pend = nullptr;
      }
      return LP_SANDWICH;
    }
    if (m.pre()) {
      a.nw_add = 1.0f;
      a.nw2 = nw2 ? nw2 : pre; a.eps = (float)m.d.norm_eps; a.mult = (float)m.d.residual_mult; a.in_scale = nw2 && m.d.logit_scale != 0.0 ? (float)m.d.logit_scale : 1.0f;
      if (pend) {
        a.y = m.y; a.xout = m.x[cur ^ 1];
        cur ^= 1;
        pend = nullptr;
      }
      return LP_PRE;
    }
    if (pend) {
      a.y = m.y; a.nw = pend; a.nw2 = nw2; a.xout = m.x[cur ^ 1]; a.eps = (float)m.d.norm_eps; a.mult = (float)m.d.residual_mult;
      pro = nw2 ? LP_HEAD : LP_RESID;
      cur ^= 1;
      pend = nullptr;
    }
    return pro;
  };
  auto mv_x = [&](int cls, const LinW& W, float* out, const float* pre, const float* nw2 = nullptr, const float* bias = nullptr, uint32_t act = 0, float cap = 0.0f) {
    LinMv a{};
    a.bias = bias; a.act = act; a.cap = cap;
    const int pro = read(a, pre, nw2);
    return mv(cls, W, out, a, pro);
  };
  for (LayeredLayer& L : m.layers) {
    float *after1 = m.ln2() ? L.post1 : L.norm1, *after2 = m.ln2() ? L.post2 : L.norm2;   // the norm that the sublayer's output waits for
    if ((rc = mv_x(LGH_K_QKV, L.in, m.cat, L.norm1, nullptr, L.in_bias))) return rc;
    if (L.latent()) {
      const LatentBufs b = latent_bufs(m, L, m.cat, m.lq);
      const uint32_t splits = latent_splits(m, L);
      if (L.d.q_rank) {
        LinMv q{};
        q.x = m.cat + L.ls.off_q; q.nw2 = L.dq_norm; q.eps = L.ls.eps; q.in_scale = 1.0f;
        if ((rc = mv(LGH_K_QKV, L.uq, m.lq, q, LP_PRE))) return rc;
      }
      if ((rc = run_k(c, LGH_K_ATTN, LGH_SYM_LATENT, (uint64_t)L.ls.heads * L.ls.rank * L.ls.dim * 2, [&] { return latent_prep_launch(L.ls, b, pos, 0, 1, m.f32, st); }))) return rc;
      if ((rc = run_k(c, LGH_K_ATTN, LGH_SYM_LATENT, mixer_bytes(c, L), [&] { return latent_attn_launch(L.ls, b, pos, 0, 1, splits, m.f32, st); }))) return rc;
      if ((rc = run_k(c, LGH_K_ATTN_COMBINE, LGH_SYM_LATENT, L.uv.bytes(), [&] {
             return latent_out_launch(L.ls, b, pos, 0, 1, splits, m.ao, 0, true, st);
           })))
        return rc;
      LinMv a{};
      a.x = m.ao;
      if ((rc = mv_end(LGH_K_WO, L.out, a, LP_COPY, after1))) return rc;
    } else if (L.tied()) {
      const TiedBufs b = tied_bufs(m, L, m.cat);
      if ((rc = run_k(c, LGH_K_ATTN, LGH_SYM_TIED, mixer_bytes(c, L), [&] { return tied_attn_launch(L.ts, b, pos, 0, 1, true, L.splits, m.f32, st); }))) return rc;
      if ((rc = run_k(c, LGH_K_ATTN_COMBINE, LGH_SYM_TIED, 0, [&] { return tied_merge_launch(L.ts, b, pos, 0, 1, L.splits, m.f32, m.ao, 0, true, st); }))) return rc;
      LinMv a{};
      a.x = m.ao;
      if ((rc = mv_end(LGH_K_WO, L.out, a, LP_COPY, after1))) return rc;
    } else if (L.glru()) {
      const GlruBufs b = glru_bufs(m, L, m.cat);
      if ((rc = run_k(c, LGH_K_ATTN, LGH_SYM_GLRU, mixer_bytes(c, L), [&] { return glru_step_launch(L.rs, b, pos, m.ao, st); }))) return rc;
      LinMv a{};
      a.x = m.ao;
      if ((rc = mv_end(LGH_K_WO, L.out, a, LP_COPY, after1))) return rc;
    } else if (L.gattn() || L.gla()) {
      const GattnBufs b = gattn_bufs(m, L, m.cat);
      const GlaBufs g = gla_bufs(m, L, m.cat, m.num);
      const GlaShape* as = L.gla() ? &L.as : nullptr;
      if (L.gattn()) {
        if ((rc = run_k(c, LGH_K_ATTN, LGH_SYM_GATTN, mixer_bytes(c, L), [&] { return gattn_attn_launch(L.gs, b, as, &g, pos, 0, 1, !b.shared, L.splits, m.f32, st); }))) return rc;
        if ((rc = run_k(c, LGH_K_ATTN_COMBINE, LGH_SYM_GATTN, 0, [&] {
               return gattn_merge_launch(L.gs, b, as, &g, L.gla_col, pos, 0, 1, L.splits, m.f32, m.ao, 0, true, st);
             })))
          return rc;
      } else {
        if ((rc = run_k(c, LGH_K_ATTN, LGH_SYM_GLA, mixer_bytes(c, L), [&] { return gla_step_launch(L.as, g, pos, 0, st); }))) return rc;
        if ((rc = run_k(c, LGH_K_ATTN_COMBINE, LGH_SYM_GLA, 0, [&] { return gla_out_launch(L.as, g, 1, m.ao, L.out.kp, true, st); }))) return rc;
      }
      LinMv a{};
      a.x = m.ao; a.bias = L.out_bias;
      if ((rc = mv_end(LGH_K_WO, L.out, a, LP_COPY, after1))) return rc;
    } else if (L.delta()) {
      const DeltaBufs b = delta_bufs(m, L, m.cat, m.num);
      if ((rc = run_k(c, LGH_K_ATTN, LGH_SYM_DELTA, mixer_bytes(c, L), [&] { return delta_step_launch(L.des, b, pos, 0, st); }))) return rc;
      LinMv a{};
      a.num = m.num; a.nw = L.gnorm; a.gate = m.cat + L.des.off_g; a.heads = L.des.heads; a.vdim = L.des.vdim; a.ldo = L.des.lv; a.eps = L.des.eps;
      if ((rc = mv_end(LGH_K_WO, L.out, a, LP_READ, after1))) return rc;
    } else {
      const MlstmBufs b = mlstm_bufs(m, L, m.cat, m.num);
      if ((rc = run_k(c, LGH_K_ATTN, LGH_SYM_MLSTM, mixer_bytes(c, L), [&] { return mlstm_step_launch(L.ms, b, pos, st); }))) return rc;
      LinMv a{};
      a.num = m.num; a.nw = L.mnorm; a.gate = m.cat + L.ms.off_g; a.heads = L.ms.heads; a.vdim = L.ms.vdim; a.ldo = L.ms.ldo; a.eps = L.ms.eps;
      if ((rc = mv_end(LGH_K_WO, L.out, a, LP_MLSTM, after1))) return rc;
    }
    if (L.moe()) {
      const RouteForm route = L.route();
      LinMv a{};                           // shared gate | up (when there is one) and the router
      const int pro = read(a, L.norm2);
      if (m.pre()) a.hout = m.h;
      a.w = L.gu.w; a.n = L.gu.n; a.paired = L.gu.paired; a.kp = L.router.kp; a.k = L.router.k; a.act = LA_SILU; a.out = m.act;
      a.w2 = L.router.w; a.n2 = L.router.n; a.out2 = m.rlogits;
      if ((rc = run_k(c, LGH_K_GATEUP, LGH_SYM_LINEAR, L.gu.bytes() + L.router.bytes(), [&] { return lin_mv_launch(pro, a, st, LS_TWO); }))) return rc;
      LinMv e{};                           // the chosen experts' gate | up
      e.x = m.dyt() || m.pre() ? m.h : m.x[cur];
      e.w2 = L.egu.w; e.n = L.egu_rows; e.paired = 1; e.kp = L.egu.kp; e.k = L.egu.k; e.act = L.d.expert_form == LGH_EXPERT_CLAMPED ? LA_CLAMPED : LA_SILU; e.limit = (float)L.d.expert_limit; e.out = m.act + L.down.kp;
      e.route = route; e.selw = m.selw;
      e.logits = m.rlogits; e.experts = L.d.experts; e.top = L.d.top; e.sel = m.sel; e.stride = (uint64_t)L.egu_rows * L.egu.kp; e.kpe = L.edown.kp;
      if ((rc = run_k(c, LGH_K_EXPERTS, LGH_SYM_LINEAR, L.egu.bytes() / L.d.experts * L.d.top, [&] { return lin_mv_launch(LP_COPY, e, st, LS_EXPERTS); }))) return rc;
      LinMv o{};
      o.x = m.act; o.w = L.down.w; o.n = m.d.width; o.kp = o.k = L.act_cols(); o.kps = L.down.kp; o.out = m.y;
      o.experts = L.d.experts; o.selw = m.selw; o.id_x = route.identity ? m.h : nullptr;
      o.w2 = L.edown.w; o.top = L.d.top; o.sel = m.sel; o.stride = (uint64_t)L.edown_rows * L.edown.kp; o.kpe = L.edown.kp;
      if (m.dyt()) o.post = post_update(c, sub++);
      else pend = after2;
      if ((rc = run_k(c, LGH_K_DOWN, LGH_SYM_LINEAR, L.down.bytes() + L.edown.bytes() / L.d.experts * L.d.top, [&] { return lin_mv_launch(LP_COPY, o, st, LS_MOE_DOWN); }))) return rc;
    } else if (L.d.ff_kind) {
      if ((rc = mv_x(LGH_K_GATEUP, L.gu, m.act, L.norm2, nullptr, nullptr, L.d.ff_kind == LGH_FF_RELU2 ? LA_RELU2 : LA_GELU))) return rc;
      LinMv a{};
      a.x = m.act;
      if ((rc = mv_end(LGH_K_DOWN, L.down, a, LP_COPY, after2))) return rc;
    }
  }
  if (mode == MODE_PREFILL && m.dyt()) return LGH_OK;
  if (mode == MODE_PREFILL && m.pre())
    return run_k(c, LGH_K_MISC, LGH_SYM_OTHER, 0, [&] { return resid_add_launch(m.x[cur], m.y, (float)m.d.residual_mult, m.d.width, m.x[cur ^ 1], st); });
  if (mode == MODE_PREFILL)
    return run_k(c, LGH_K_MISC, LGH_SYM_OTHER, 0, [&] {
      return resid_norm_out_launch(m.x[cur], m.y, pend, (float)m.d.norm_eps, (float)m.d.residual_mult, m.d.width, m.x[cur ^ 1], st);
    });
  if ((rc = mv_x(LGH_K_OUTPUT, m.head, c->logits, nullptr, m.final_norm, nullptr, 0, (float)m.d.logit_cap))) return rc;
  if (mode == MODE_GREEDY)
    return run_k(c, LGH_K_ARGMAX, LGH_SYM_ARGMAX, (uint64_t)m.d.vocab_size * 4, [&] {
      return argmax_launch(c->logits, m.d.vocab_size, c->amax_v, c->amax_i, c->state, c->tok_log, st);
    });
  return LGH_OK;
}

uint64_t layered_step_bytes(const lgh_ctx* c) {
  const LayeredModel& m = *c->lm;
  uint64_t b = (uint64_t)m.d.width * (m.bigram ? 4 : 2) + m.head.bytes() + (uint64_t)m.d.vocab_size * 4 + m.d.width * 4;
  for (const LayeredLayer& L : m.layers) {
    b += L.in.bytes() + L.out.bytes() + mixer_bytes(c, L) + (uint64_t)m.d.width * 4;
    if (L.latent()) b += L.uk.bytes() + L.uv.bytes() + L.uq.bytes();
    if (m.ln2()) b += (uint64_t)m.d.width * (L.d.ff_kind ? 8 : 4);
    if (L.d.ff_kind) b += L.gu.bytes() + L.down.bytes() + (uint64_t)m.d.width * 4;
    if (L.moe()) b += L.router.bytes() + (L.egu.bytes() + L.edown.bytes()) / L.d.experts * L.d.top;
  }
  return b;
}

// ------------------------------------------------------------------------------------------------
// blocks of tokens
// ------------------------------------------------------------------------------------------------
static int block_ensure(lgh_ctx* c) {
  LayeredModel& m = *c->lm;
  if (m.blk_ready) return LGH_OK;
  const lgh_layered_desc& d = m.d;
  m.blk = std::min(kBlockTokens, d.max_seq_len);
  uint32_t heads = 0, hdim = 0;
  for (auto& L : m.layers)
    if (L.mlstm()) { heads = std::max(heads, L.ms.heads); hdim = std::max(hdim, L.ms.heads * L.ms.dim); }
    else if (L.gla()) heads = std::max(heads, L.as.heads);
  const size_t moe_tiles = moe_max_tiles(m.blk * m.max_top, std::max(m.max_experts, 1u), 16);
  const size_t B = m.blk, chunks = (B + 63) / 64, Bc = chunks * 64, el = m.el();
  struct { void** p; size_t n; } bufs[] = {
      {(void**)&m.bx, B * d.width * 4}, {&m.bxa, B * up(d.width, 64) * el}, {(void**)&m.by, B * up(d.width, 4) * 4},
      {(void**)&m.bcat, (B * m.max_cat + kMlstmRowSlack) * 4}, {&m.bao, B * m.max_ao * el}, {&m.bact, B * m.max_act * el},
      {(void**)&m.bnum, Bc * m.max_num * 4}, {(void**)&m.blq, B * m.max_lq * 4}, {&m.blqa, B * m.max_qrank * el},
      {(void**)&m.bdq, Bc * m.max_dqk * 4}, {(void**)&m.bdk, Bc * m.max_dqk * 4}, {(void**)&m.bdv, Bc * m.max_dv * 4}, {(void**)&m.bdu, Bc * m.max_dv * 4},
      {(void**)&m.bdw, Bc * m.max_dw * 4}, {(void**)&m.bdp, Bc * m.max_dw * 4}, {(void**)&m.bdwge, Bc * m.max_dheads * 4}, {(void**)&m.bdcd, chunks * m.max_dheads * 4},
      {(void**)&m.ba, chunks * heads * 4096 * 4}, {(void**)&m.bu, heads * Bc * 8}, {(void**)&m.bmx, heads * Bc * 8},
      {(void**)&m.bdec, heads * Bc * 4}, {(void**)&m.bwgt, heads * Bc * 4}, {(void**)&m.bcdec, heads * chunks * 4}, {(void**)&m.bnk, chunks * hdim * 4},
      {(void**)&m.brec, B * m.max_rec * 2 * 4}, {(void**)&m.brsum, (chunks * 2 + 1) * m.max_rec * 4},
      {(void**)&m.bqk, m.max_gla ? (Bc * m.max_gla * 2 + kMlstmRowSlack) * 4 : 0}, {(void**)&m.bgdec, m.max_gla ? (chunks * m.max_gla + kMlstmRowSlack) * 4 : 0},
      {(void**)&m.bx2, m.dyt() ? B * d.width * 4 : 0}, {(void**)&m.tails, m.hist_floats() * 4}, {&m.btq, B * m.max_tied_q * el},
      {(void**)&m.bpair, B * m.max_top * up(d.width, 4) * 4}, {&m.bpact, B * m.max_pair_act * el},
      {(void**)&m.bsel, B * m.max_top * 4}, {(void**)&m.bselw, B * m.max_top * 4}, {(void**)&m.bslot, B * m.max_top * 4}, {(void**)&m.bsrc, B * m.max_top * 4},
      {(void**)&m.broww, B * m.max_top * 4}, {(void**)&m.bseg, (size_t)(m.max_experts + 1) * 4}, {(void**)&m.btile_e, m.max_top ? moe_tiles * 4 : 0},
      {(void**)&m.btile_row, m.max_top ? moe_tiles * 4 : 0},
      {(void**)&m.btok, B * 4}, {(void**)&m.brows, B * 4}, {&m.bla, (size_t)kLogitRows * up(d.width, 64) * el},
      {(void**)&m.blogits, (size_t)kLogitRows * up(d.vocab_size, 4) * 4},
  };
  int rc;
  for (auto& b : bufs)
    if ((rc = zeroed(c, b.p, b.n, &c->stats.scratch_bytes))) return rc;
  L_TRY(c, LGH_OPERATION_FAILED, hipStreamSynchronize(c->stream));
  m.blk_ready = true;
  return LGH_OK;
}

static int block_gemm(lgh_ctx* c, int cls, const LinW& W, int epi, const void* x, uint32_t ldx, void* out, uint32_t ldo, uint32_t M, const float* bias = nullptr, float cap = 0.0f) {
  LinGemm g{};
  g.bias = bias; g.cap = cap;
  g.w = W.w; g.x = x; g.out = out; g.n = W.n; g.np = W.np(); g.kp = W.kp; g.ldx = ldx; g.ldo = ldo; g.M = M;
  return run_k(c, cls, LGH_SYM_LINEAR, W.bytes(), [&] { return lin_gemm_launch(epi, c->lm->f32, g, c->stream); });
}

// a buffer of the expanded path, grown when the context does (zeroed: the padding of a key tile must be finite)
static int grow(lgh_ctx* c, void** p, size_t* have, size_t need) {
  if (*have >= need) return LGH_OK;
  L_TRY(c, LGH_OPERATION_FAILED, hipStreamSynchronize(c->stream));
  if (*p) dev_free_tracked(c, *p);
  c->stats.scratch_bytes -= *have;
  *p = nullptr;
  *have = 0;
  if (int rc = zeroed(c, p, need, &c->stats.scratch_bytes)) return rc;
  *have = need;
  return LGH_OK;
}

// portions from this many tokens on form keys and values per head when the context is not much longer than they are
constexpr uint32_t kExpandTokens = 64;

static int block_latent(lgh_ctx* c, LayeredLayer& L, uint32_t pos0, uint32_t M) {
  LayeredModel& m = *c->lm;
  hipStream_t st = c->stream;
  int rc;
  LatentFlash& f = m.fl;
  if (L.d.q_rank) {
    if ((rc = run_k(c, LGH_K_QKV, LGH_SYM_OTHER, 0, [&] {
           return rms_cols_launch(m.bcat + L.ls.off_q, L.ls.ldcat, L.dq_norm, L.ls.eps, L.d.q_rank, M, m.blqa, L.uq.kp, m.f32, st);
         })))
      return rc;
    if ((rc = block_gemm(c, LGH_K_QKV, L.uq, LE_F32, m.blqa, L.uq.kp, m.blq, L.ls.ldq, M))) return rc;
  }
  f.base = latent_key_start(L.ls, pos0) / 64 * 64;
  if (M >= kExpandTokens && pos0 - f.base <= 64 * M && latent_flash_shape(L.ls, &f.dq, &f.dvp)) {
    const uint32_t kv = pos0 - f.base + M, H = L.ls.heads;   // positions from the first visible tile on
    f.Mcap = m.blk;
    f.Tcap = up(kv, 1024);
    if ((rc = grow(c, &f.q, &m.fl_q_bytes, (size_t)H * f.Mcap * f.dq * m.el())) || (rc = grow(c, &f.k, &m.fl_k_bytes, (size_t)H * f.Tcap * f.dq * m.el())) ||
        (rc = grow(c, &f.vt, &m.fl_v_bytes, (size_t)H * f.dvp * f.Tcap * m.el())))
      return rc;
    const LatentBufs b = latent_bufs(m, L, m.bcat, m.blq);
    if ((rc = run_k(c, LGH_K_EXPAND, LGH_SYM_LATENT, 0, [&] { return latent_flash_prep_launch(L.ls, b, f, pos0, M, m.f32, st); }))) return rc;
    LinGemm g{};
    g.x = (const uint8_t*)L.cache + (size_t)f.base * L.ls.ldc * m.el(); g.ldx = L.ls.ldc; g.M = kv;
    g.w = L.uk.w; g.n = L.uk.n; g.np = L.uk.np(); g.kp = L.uk.kp; g.out = f.k; g.ldo = f.dq; g.hd = L.ls.dim; g.tcap = f.Tcap;
    if ((rc = run_k(c, LGH_K_EXPAND, LGH_SYM_LINEAR, L.uk.bytes(), [&] { return lin_gemm_launch(LE_HEADS, m.f32, g, st); }))) return rc;
    g.w = L.uv.w; g.n = L.uv.n; g.np = L.uv.np(); g.kp = L.uv.kp; g.out = f.vt; g.ldo = (uint32_t)f.Tcap; g.hd = L.ls.vdim; g.hrows = f.dvp;
    if ((rc = run_k(c, LGH_K_EXPAND, LGH_SYM_LINEAR, L.uv.bytes(), [&] { return lin_gemm_launch(LE_HEADS_T, m.f32, g, st); }))) return rc;
    return run_k(c, LGH_K_ATTN, LGH_SYM_LATENT, 0, [&] { return latent_flash_launch(L.ls, b, f, pos0, M, m.f32, m.bao, L.out.kp, st); });
  }
  // absorbed, as many tokens at a time as their (token, head) rows fit the buffers
  const uint32_t step = std::max(1u, kLatAbsorbRows / L.ls.heads);
  for (uint32_t t = 0; t < M; t += step) {
    const uint32_t n = std::min(step, M - t), p = pos0 + t;
    const uint32_t splits = std::max(1u, std::min(m.n_splits, 512u / ((n * L.ls.heads + 15) / 16)));
    const LatentBufs b = latent_bufs(m, L, m.bcat + (size_t)t * L.ls.ldcat, m.blq + (L.d.q_rank ? (size_t)t * L.ls.ldq : 0));
    if ((rc = run_k(c, LGH_K_ATTN, LGH_SYM_LATENT, 0, [&] { return latent_prep_launch(L.ls, b, nullptr, p, n, m.f32, st); }))) return rc;
    if ((rc = run_k(c, LGH_K_ATTN, LGH_SYM_LATENT, 0, [&] { return latent_attn_launch(L.ls, b, nullptr, p, n, splits, m.f32, st); }))) return rc;
    if ((rc = run_k(c, LGH_K_ATTN_COMBINE, LGH_SYM_LATENT, 0, [&] {
           return latent_out_launch(L.ls, b, nullptr, p, n, splits, (uint8_t*)m.bao + (size_t)t * L.out.kp * m.el(), L.out.kp, m.f32, st);
         })))
      return rc;
  }
  return LGH_OK;
}

static int block_tied(lgh_ctx* c, LayeredLayer& L, uint32_t pos0, uint32_t M) {
  LayeredModel& m = *c->lm;
  hipStream_t st = c->stream;
  int rc;
  TiedBufs b = tied_bufs(m, L, m.bcat);
  const bool flash = M > kTiedShort;
  if (flash) { b.q = m.btq; b.Mcap = m.blk; }
  if ((rc = run_k(c, LGH_K_EXPAND, LGH_SYM_TIED, 0, [&] { return tied_prep_launch(L.ts, b, pos0, M, m.f32, st); }))) return rc;
  if (flash) return run_k(c, LGH_K_ATTN, LGH_SYM_TIED, 0, [&] { return tied_flash_launch(L.ts, b, pos0, M, m.f32, m.bao, L.out.kp, st); });
  const uint32_t splits = tied_splits(L.ts, m.d.max_seq_len, M, m.f32, m.forced_splits);
  if ((rc = run_k(c, LGH_K_ATTN, LGH_SYM_TIED, 0, [&] { return tied_attn_launch(L.ts, b, nullptr, pos0, M, false, splits, m.f32, st); }))) return rc;
  return run_k(c, LGH_K_ATTN_COMBINE, LGH_SYM_TIED, 0, [&] { return tied_merge_launch(L.ts, b, nullptr, pos0, M, splits, m.f32, m.bao, L.out.kp, m.f32, st); });
}

// gated attention and / or gated linear attention of a block, side by side in the output product's input
static int block_gattn(lgh_ctx* c, LayeredLayer& L, uint32_t pos0, uint32_t M) {
  LayeredModel& m = *c->lm;
  hipStream_t st = c->stream;
  int rc;
  if (L.gattn()) {
    GattnBufs b = gattn_bufs(m, L, m.bcat);
    const bool flash = M > kGattnShort && L.gs.dp <= kGattnFlashDim;
    if (flash) { b.q = m.btq; b.Mcap = m.blk; }
    if ((rc = run_k(c, LGH_K_EXPAND, LGH_SYM_GATTN, 0, [&] { return gattn_prep_launch(L.gs, b, pos0, M, m.f32, st); }))) return rc;
    if (flash) {
      if ((rc = run_k(c, LGH_K_ATTN, LGH_SYM_GATTN, 0, [&] { return gattn_flash_launch(L.gs, b, pos0, M, m.f32, m.bao, L.out.kp, st); }))) return rc;
    } else {
      for (uint32_t t = 0; t < M; t += kGattnShort) {
        const uint32_t n = std::min(kGattnShort, M - t), splits = gattn_splits(L.gs, m.d.max_seq_len, n, m.f32, m.forced_splits);
        b.cat = m.bcat + (size_t)t * L.gs.ldcat;
        if ((rc = run_k(c, LGH_K_ATTN, LGH_SYM_GATTN, 0, [&] { return gattn_attn_launch(L.gs, b, nullptr, nullptr, nullptr, pos0 + t, n, false, splits, m.f32, st); }))) return rc;
        if ((rc = run_k(c, LGH_K_ATTN_COMBINE, LGH_SYM_GATTN, 0, [&] {
               return gattn_merge_launch(L.gs, b, nullptr, nullptr, 0, nullptr, pos0 + t, n, splits, m.f32, (uint8_t*)m.bao + (size_t)t * L.out.kp * m.el(), L.out.kp, m.f32, st);
             })))
          return rc;
      }
    }
  }
  if (L.gla()) {
    const GlaBufs g = gla_bufs(m, L, m.bcat, m.bnum);
    if ((rc = run_k(c, LGH_K_ATTN, LGH_SYM_GLA, 0, [&] { return gla_block_launch(L.as, g, pos0, M, st); }))) return rc;
    if ((rc = run_k(c, LGH_K_ATTN_COMBINE, LGH_SYM_GLA, 0, [&] { return gla_out_launch(L.as, g, M, (uint8_t*)m.bao + (size_t)L.gla_col * m.el(), L.out.kp, m.f32, st); }))) return rc;
  }
  return LGH_OK;
}

// routed experts of a block: the pairs' outputs -> m.bpair, rows m.bslot; the shared expert -> m.by
static int block_moe(lgh_ctx* c, LayeredLayer& L, uint32_t ldx, uint32_t ldy, uint32_t M) {
  LayeredModel& m = *c->lm;
  hipStream_t st = c->stream;
  int rc;
  const uint32_t E = L.d.experts, rows = M * L.d.top;
  MoeRoute r{};
  r.x = m.bxa; r.ldx = ldx; r.router = L.router.w; r.kp = L.router.kp; r.M = M; r.experts = E; r.top = L.d.top; r.bm = lin_group_rows(rows, std::min(rows, E));
  r.sel = m.bsel; r.w = m.bselw; r.seg = m.bseg; r.tile_e = m.btile_e; r.tile_row = m.btile_row; r.slot = m.bslot; r.src = m.bsrc; r.roww = m.broww;
  r.tiles = moe_max_tiles(rows, E, r.bm);
  r.route = L.route();
  if ((rc = run_k(c, LGH_K_ROUTER, LGH_SYM_OTHER, 0, [&] { return moe_route_launch(r, m.f32, st); }))) return rc;
  LinGemm g{};
  g.grp.seg = r.seg; g.grp.tile_e = r.tile_e; g.grp.tile_row = r.tile_row; g.grp.tiles = r.tiles; g.grp.bm = r.bm;
  g.w = L.egu.w; g.n = g.np = L.egu_rows; g.kp = L.egu.kp; g.M = rows; g.x = m.bxa; g.ldx = ldx; g.out = m.bpact; g.ldo = L.edown.kp;
  g.grp.src = r.src; g.grp.scale = r.roww; g.grp.stride = (uint64_t)L.egu_rows * L.egu.kp;
  g.grp.limit = (float)L.d.expert_limit;
  const int epi = L.d.expert_form == LGH_EXPERT_CLAMPED ? LE_CLAMPED : LE_SWIGLU;
  if ((rc = run_k(c, LGH_K_EXPERTS, LGH_SYM_LINEAR, L.egu.bytes(), [&] { return lin_gemm_launch(epi, m.f32, g, st); }))) return rc;
  g.w = L.edown.w; g.n = m.d.width; g.np = L.edown_rows; g.kp = L.edown.kp; g.x = m.bpact; g.ldx = L.edown.kp; g.out = m.bpair; g.ldo = ldy;
  g.grp.src = nullptr; g.grp.scale = nullptr; g.grp.stride = (uint64_t)L.edown_rows * L.edown.kp;
  if ((rc = run_k(c, LGH_K_DOWN, LGH_SYM_LINEAR, L.edown.bytes(), [&] { return lin_gemm_launch(LE_F32, m.f32, g, st); }))) return rc;
  if (L.d.shared_ff) {
    if ((rc = block_gemm(c, LGH_K_GATEUP, L.gu, LE_SWIGLU, m.bxa, ldx, m.bact, L.down.kp, M))) return rc;
    if ((rc = block_gemm(c, LGH_K_DOWN, L.down, LE_F32, m.bact, L.down.kp, m.by, ldy, M))) return rc;
  }
  return LGH_OK;
}

static int block_pass(lgh_ctx* c, const uint32_t* tokens, uint32_t M, const uint32_t* want, uint32_t n_want, float* logits_out) {
  LayeredModel& m = *c->lm;
  const lgh_layered_desc& d = m.d;
  hipStream_t st = c->stream;
  const uint32_t pos0 = (uint32_t)c->pos, ldx = up(d.width, 64), ldy = up(d.width, 4);
  const float eps = (float)d.norm_eps, mult = (float)d.residual_mult;
  int rc;
  L_TRY(c, LGH_OPERATION_FAILED, hipMemcpyAsync(m.btok, tokens, (size_t)M * 4, hipMemcpyHostToDevice, st));
  if ((rc = run_k(c, LGH_K_EMBED, LGH_SYM_EMBED, (uint64_t)M * d.width * 4, [&] {
         return layered_embed_block_launch(embed_args(m), m.btok, pos0, M, m.bx, m.bxa, ldx, m.f32, st);
       })))
    return rc;
  float* xs = m.bx;                        // the residual stream
  uint32_t sub = 0;
  // LGH_RESIDUAL_SANDWICH_DYT: the sublayer's output into the stream, then the next sublayer's input; from_embed: the latter alone
  auto resid_dyt = [&](bool from_embed, const LayeredLayer* moe) {
    DytBlock b{};
    b.x = xs; b.width = d.width; b.M = M; b.pos0 = pos0; b.mult = mult; b.ldx = ldx;
    if (!from_embed) {
      b.xout = xs == m.bx ? m.bx2 : m.bx;
      b.post = dyt_w(m.subs[sub++].post);
      if (!moe || moe->d.shared_ff) { b.y = m.by; b.ldy = ldy; }
      if (moe) { b.pairs = m.bpair; b.ldp = ldy; b.slot = m.bslot; b.top = moe->d.top; }
      xs = b.xout;
    }
    if (sub < m.n_sub) {
      b.next = dyt_w(m.subs[sub].pre); b.conv = conv_w(m, sub); b.xa = m.bxa;
      b.tail = m.hist_floats() ? m.tails + (size_t)sub * (d.conv_taps - 1) * d.width : nullptr;
    }
    return run_k(c, LGH_K_MISC, LGH_SYM_OTHER, (uint64_t)M * d.width * 14, [&] { return dyt_block_launch(b, m.f32, st); });
  };
  if (m.dyt() && (rc = resid_dyt(true, nullptr))) return rc;
  // LGH_RESIDUAL_PRE_RMS: the sublayer's output into the stream, then its norm in front of the next sublayer (nw NULL: there is none)
  auto resid_pre = [&](const float* nw, bool from_embed, const LayeredLayer* moe) {
    PreBlock b{};
    b.x = m.bx; b.width = d.width; b.M = M; b.mult = mult; b.eps = eps; b.nw = nw; b.xa = m.bxa; b.ldx = ldx;
    if (!from_embed && (!moe || moe->d.shared_ff)) { b.y = m.by; b.ldy = ldy; }
    if (moe) { b.pairs = m.bpair; b.ldp = ldy; b.slot = m.bslot; b.selw = m.bselw; b.top = moe->d.top; }
    return run_k(c, LGH_K_MISC, LGH_SYM_OTHER, (uint64_t)M * d.width * 14, [&] { return pre_block_launch(b, m.f32, st); });
  };
  if (m.pre() && (rc = resid_pre(m.layers[0].norm1, true, nullptr))) return rc;
  // LGH_RESIDUAL_SANDWICH_LN: the sublayer's output through the norm behind it (NULL: there is no output yet), then the next sublayer's norm
  auto resid_ln = [&](const float* post, const float* nw) {
    LnBlock b{};
    b.x = m.bx; b.width = d.width; b.M = M; b.mult = mult; b.eps = eps; b.nw = nw; b.xa = m.bxa; b.ldx = ldx;
    if (post) { b.y = m.by; b.ldy = ldy; b.pw = post; }
    return run_k(c, LGH_K_MISC, LGH_SYM_OTHER, (uint64_t)M * d.width * 14, [&] { return ln_block_launch(b, m.f32, st); });
  };
  if (m.ln2() && (rc = resid_ln(nullptr, m.layers[0].norm1))) return rc;
  const float* next = nullptr;             // the norm in front of the sublayer that follows
  auto resid = [&](const float* nw, const LayeredLayer* moe = nullptr) -> int {
    if (m.pre()) return resid_pre(next, false, moe);
    if (m.ln2()) return resid_ln(nw, next);
    if (m.dyt()) return resid_dyt(false, moe);
    if (moe && (rc = run_k(c, LGH_K_MISC, LGH_SYM_OTHER, 0, [&] {
                  return pair_sum_launch(m.by, ldy, m.bpair, ldy, m.bslot, moe->d.top, d.width, M, moe->d.shared_ff != 0, st);
                })))
      return rc;
    return run_k(c, LGH_K_MISC, LGH_SYM_OTHER, (uint64_t)M * d.width * 14, [&] {
      return resid_norm_launch(m.bx, m.by, ldy, nw, eps, mult, d.width, M, m.bxa, ldx, m.f32, st);
    });
  };
  for (uint32_t li = 0; li < d.num_layers; li++) {
    LayeredLayer& L = m.layers[li];
    const float* after = li + 1 < d.num_layers ? m.layers[li + 1].norm1 : nullptr;
    if ((rc = block_gemm(c, LGH_K_QKV, L.in, LE_F32, m.bxa, ldx, m.bcat, L.in.n, M, L.in_bias))) return rc;
    if (L.latent()) {
      if ((rc = block_latent(c, L, pos0, M))) return rc;
    } else if (L.delta()) {
      const DeltaBufs b = delta_bufs(m, L, m.bcat, m.bnum);
      if ((rc = run_k(c, LGH_K_ATTN, LGH_SYM_DELTA, 0, [&] { return delta_block_launch(L.des, b, pos0, M, st); }))) return rc;
      if ((rc = run_k(c, LGH_K_ATTN_COMBINE, LGH_SYM_DELTA, 0, [&] { return delta_out_launch(L.des, b, pos0, M, m.bao, L.out.kp, m.f32, st); }))) return rc;
    } else if (L.tied()) {
      if ((rc = block_tied(c, L, pos0, M))) return rc;
    } else if (L.glru()) {
      const GlruBufs b = glru_bufs(m, L, m.bcat);
      if ((rc = run_k(c, LGH_K_ATTN, LGH_SYM_GLRU, 0, [&] { return glru_block_launch(L.rs, b, pos0, M, m.f32, m.bao, L.out.kp, st); }))) return rc;
    } else if (L.gattn() || L.gla()) {
      if ((rc = block_gattn(c, L, pos0, M))) return rc;
    } else {
      const MlstmBufs b = mlstm_bufs(m, L, m.bcat, m.bnum);
      if ((rc = run_k(c, LGH_K_ATTN, LGH_SYM_MLSTM, 0, [&] { return mlstm_block_launch(L.ms, b, pos0, M, st); }))) return rc;
      if ((rc = run_k(c, LGH_K_ATTN_COMBINE, LGH_SYM_MLSTM, 0, [&] { return mlstm_out_launch(L.ms, b, M, m.bao, L.out.kp, m.f32, st); }))) return rc;
    }
    if ((rc = block_gemm(c, LGH_K_WO, L.out, LE_F32, m.bao, L.out.kp, m.by, ldy, M, L.out_bias))) return rc;
    next = L.d.ff_kind ? L.norm2 : after;
    if ((rc = resid(m.ln2() ? L.post1 : L.norm1))) return rc;
    next = after;
    if (L.moe()) {
      if ((rc = block_moe(c, L, ldx, ldy, M))) return rc;
      if ((rc = resid(L.norm2, &L))) return rc;
    } else if (L.d.ff_kind) {
      if ((rc = block_gemm(c, LGH_K_GATEUP, L.gu, L.d.ff_kind == LGH_FF_RELU2 ? LE_RELU2 : LE_GEGLU, m.bxa, ldx, m.bact, L.down.kp, M))) return rc;
      if ((rc = block_gemm(c, LGH_K_DOWN, L.down, LE_F32, m.bact, L.down.kp, m.by, ldy, M))) return rc;
      if ((rc = resid(m.ln2() ? L.post2 : L.norm2))) return rc;
    }
    if (m.tap && m.tap_tokens == M)
      L_TRY(c, LGH_OPERATION_FAILED, hipMemcpyAsync(m.tap_buf + (size_t)li * M * d.width, xs, (size_t)M * d.width * 4, hipMemcpyDeviceToDevice, st));
  }
  L_TRY(c, LGH_OPERATION_FAILED, hipMemcpyAsync(c->hidden, xs + (size_t)(M - 1) * d.width, (size_t)d.width * 4, hipMemcpyDeviceToDevice, st));
  if (m.hist_floats() && (rc = run_k(c, LGH_K_MISC, LGH_SYM_OTHER, 0, [&] {
                            return conv_store_launch(m.tails, m.hist, m.n_sub, d.conv_taps, d.width, pos0, M, st);
                          })))
    return rc;
  const uint32_t ldl = up(d.vocab_size, 4);
  for (uint32_t w = 0; w < n_want; w += kLogitRows) {
    const uint32_t n = std::min(kLogitRows, n_want - w);
    L_TRY(c, LGH_OPERATION_FAILED, hipMemcpyAsync(m.brows, want + w, (size_t)n * 4, hipMemcpyHostToDevice, st));
    if ((rc = run_k(c, LGH_K_MISC, LGH_SYM_OTHER, 0, [&] {
           if (m.pre()) return final_rms_rows_launch(xs, m.brows, n, m.final_norm, eps, d.logit_scale != 0.0 ? (float)d.logit_scale : 1.0f, d.width, m.bla, ldx, m.f32, st);
           return m.dyt() ? final_dyt_rows_launch(xs, m.brows, n, dyt_w(m.final_dyt), d.width, m.bla, ldx, m.f32, st)
                          : final_norm_rows_launch(xs, m.brows, n, m.final_norm, eps, d.width, m.bla, ldx, m.f32, st);
         })))
      return rc;
    if ((rc = block_gemm(c, LGH_K_OUTPUT, m.head, LE_F32, m.bla, ldx, m.blogits, ldl, n, nullptr, (float)d.logit_cap))) return rc;
    L_TRY(c, LGH_OPERATION_FAILED, hipMemcpy2DAsync(logits_out + (size_t)w * d.vocab_size, (size_t)d.vocab_size * 4, m.blogits, (size_t)ldl * 4,
                                                    (size_t)d.vocab_size * 4, n, hipMemcpyDeviceToHost, st));
    L_TRY(c, LGH_OPERATION_FAILED, hipStreamSynchronize(st));
  }
  c->pos += M;
  c->stats.tokens_processed += M;
  L_TRY(c, LGH_OPERATION_FAILED, hipMemsetD32Async((hipDeviceptr_t)(c->state + ST_NEXT), (int)c->pos, 1, st));
  L_TRY(c, LGH_OPERATION_FAILED, hipStreamSynchronize(st));   // the caller's tokens / want are free again
  return c->profiling ? drain_prof(c) : LGH_OK;
}

int layered_block(lgh_ctx* c, const uint32_t* tokens, size_t n, const uint32_t* want, size_t n_want, float* logits_out) {
  LayeredModel& m = *c->lm;
  int rc = block_ensure(c);
  if (rc) return rc;
  if (m.tap) {
    m.tap_tokens = 0;
    if (m.tap_buf) dev_free_tracked(c, m.tap_buf);
    m.tap_buf = nullptr;
    if (n <= m.blk) {
      if ((rc = dev_alloc(c, (void**)&m.tap_buf, (size_t)m.d.num_layers * n * m.d.width * 4))) return rc;
      m.tap_tokens = (uint32_t)n;
    }
  }
  size_t w = 0;
  std::vector<uint32_t> local;
  for (size_t t = 0; t < n; t += m.blk) {
    const uint32_t M = (uint32_t)std::min<size_t>(m.blk, n - t);
    local.clear();
    const size_t w0 = w;
    while (w < n_want && want[w] < t + M) local.push_back((uint32_t)(want[w++] - t));
    if ((rc = block_pass(c, tokens + t, M, local.data(), (uint32_t)local.size(), logits_out ? logits_out + w0 * m.d.vocab_size : nullptr))) return rc;
  }
  return LGH_OK;
}

extern "C" int lgh_set_layer_tap(lgh_ctx* c, int on) {
  if (!c) return LGH_INVALID_ARGUMENT;
  if (!c->lm) return fail(c, LGH_UNSUPPORTED, "only models described layer by layer have a layer tap");
  c->lm->tap = on != 0;
  c->lm->tap_tokens = 0;
  return LGH_OK;
}

extern "C" int lgh_read_layers(lgh_ctx* c, float* out, size_t n_floats) {
  if (!c || !out) return LGH_INVALID_ARGUMENT;
  if (!c->lm || !c->lm->tap_tokens) return fail(c, LGH_INVALID_ARGUMENT, "no portion was run with the layer tap on");
  const size_t n = (size_t)c->lm->d.num_layers * c->lm->tap_tokens * c->lm->d.width;
  if (n_floats != n) return fail(c, LGH_SHAPE_MISMATCH, "expected " + std::to_string(n) + " floats");
  if (hipSetDevice(c->device) != hipSuccess) return fail(c, LGH_NOT_AVAILABLE, "hipSetDevice failed");
  L_TRY(c, LGH_OPERATION_FAILED, hipMemcpyAsync(out, c->lm->tap_buf, n * 4, hipMemcpyDeviceToHost, c->stream));
  L_TRY(c, LGH_OPERATION_FAILED, hipStreamSynchronize(c->stream));
  return LGH_OK;
}
