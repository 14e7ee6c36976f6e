// layered_model.cpp -- layered models (layered.h) behind the model-family table: weights into HBM, the sequences' state, steps.
//
// A parallel layer is five launches and its mixers': [residual sum + norm] -> one matrix product for everything that reads the norm
// (the mixers' projections, gates, the router) -> mixers -> their output products -> experts (up, down).  A sandwich layer has a second
// [residual sum + norms + convolution] between its mixer and a dense feed-forward.  A step's tokens are packed without padding; every
// sequence owns an arena whose size does not depend on its length (one chunk of keys and values, a window of latents, recurrent
// state, convolution inputs).  Steps of at most 16 single tokens run on the kernels for few rows, from a captured graph.
#include "layered.h"

#include <math.h>
#include <stdlib.h>
#include <string.h>

#include <algorithm>

namespace {

enum { FEW = 16, LOGIT_ROWS = 128, MIX_PARTS = 4, MIX_PARTS_FEW = 8 };

size_t up(size_t v, size_t a) { return (v + a - 1) / a * a; }

struct ConvW {           // a sandwich layer's convolution in front of a sublayer
  float *w = nullptr, *mu = nullptr;
  int n_mix = 0;         // blends with the previous token (wkv), in the order of the projections
  size_t off_in = 0, off_prev = 0;
};
struct LayerW {
  float* norm = nullptr;
  float *post = nullptr, *ff_norm = nullptr, *ff_post = nullptr;
  ConvW conv, ff_conv;
  PackedMat proj;        // every product of the norm's output: wide segments (activation type), then 32-bit segments
  int n_wide = 0;        // columns of the wide part (multiple of 64)
  // attention
  int a_q = 0, a_k = 0, a_v = 0;
  float* freq = nullptr;
  float rot_amp = 1.f;
  PackedMat a_o;
  size_t off_k = 0, off_v = 0;
  // mLSTM
  int m_q = 0, m_k = 0, m_v = 0, m_g = 0, m_i = 0, m_f = 0;
  float *m_bi = nullptr, *m_bf = nullptr, *m_norm = nullptr;
  PackedMat m_o;
  size_t off_ms = 0, off_mn = 0, off_mm = 0;
  // delta rule
  int d_q = 0, d_k = 0, d_v = 0, d_low = 0, d_b = 0;
  int low_a = 0, low_g = 0;  // ranks of the low-rank pairs
  PackedMat d_low2, d_o;  // both second halves of the low-rank pairs, block-diagonal
  float *d_conv = nullptr, *d_rate = nullptr, *d_dt = nullptr, *d_norm = nullptr;
  size_t off_ds = 0, off_dc = 0;
  int d_a = 0, d_g = 0;   // (decay per head, gate by silu)
  // wkv
  int w_r = 0, w_k = 0, w_v = 0, w_g = 0, w_low = 0, seg = 0;  // seg: features per blend
  PackedMat w_low2, w_o;
  float *w_w0 = nullptr, *w_u = nullptr, *w_norm = nullptr;
  size_t off_ws = 0;
  // latent attention
  int l_q = 0, l_kv = 0;
  int dim_p = 0, rot_p = 0, vdim_p = 0, rank_p = 0;
  float *l_qn = nullptr, *l_kvn = nullptr;
  PackedMat l_uq, l_ukv, l_abs, l_o;  // l_abs: W_uk transposed per head, queries into the latent space
  size_t off_lc = 0;
  // dense feed-forward
  PackedMat ff_up, ff_down;
  float ff_pos = 0.f, ff_neg = 0.f;
  float *pair_a = nullptr, *pair_b = nullptr;
  int router = 0;
  ExpertMat e_up{}, e_down{};
};

struct Seq {
  char* base = nullptr;
  bool live = false;
  int pos = 0, flip = 0;
};

// one buffer of pass descriptors: pinned host side and device side, `cap` rows
struct DescBuf {
  char *host = nullptr, *dev = nullptr;
  int cap = 0;
  size_t o_tok = 0, o_row = 0, o_want = 0, o_tile = 0, o_chunk = 0, o_single = 0, bytes = 0;
};

struct Graph {
  hipGraphExec_t exec = nullptr;
  bool primed = false;
};

enum { OUT_NONE = 0, OUT_LOGITS = 1, OUT_ARGMAX = 2, OUT_SAMPLE = 3 };

struct LayeredModel : ModelHead {
  LayeredSpec s;
  bool f32 = false;
  int piece = 2048;
  bool use_graph = true, fused_decode = true, trace = false;
  std::vector<void*> dev;           // device allocations of the model
  double weight_bytes = 0, scratch_bytes = 0;
  uint16_t* embed = nullptr;
  float* final_norm = nullptr;
  PackedMat head;
  std::vector<LayerW> L;
  // sequences
  size_t seq_bytes = 0;
  std::vector<Seq> seqs;
  std::vector<void*> slabs;
  double cache_bytes = 0;
  int32_t own_seq = -1;             // dsk_forward / dsk_hydrate: the model's own sequence
  // workspaces
  int ldw = 0, ldf = 0, h_ld = 0, mix_ld = 0, out_ld = 0, low_ld = 0, hid_ld = 0, y_ld = 0, ld_logits = 0, max_tiles = 0, slots = 0;
  float* x = nullptr;
  char *h = nullptr, *hw = nullptr, *wide = nullptr, *out_a = nullptr, *out_b = nullptr, *qb = nullptr, *kb = nullptr, *vb = nullptr, *hidden = nullptr, *y = nullptr;
  float *narrow = nullptr, *mix_a = nullptr, *mix_b = nullptr, *low = nullptr, *dq = nullptr, *dk = nullptr, *dv = nullptr, *dg = nullptr, *db = nullptr, *o = nullptr;
  int mix_parts[2] = {1, 1};        // of the products that wrote mix_a and mix_b last
  size_t mix_stride = 0;
  // sandwich layers, latent attention
  float *h_f = nullptr, *turn = nullptr, *lat_part = nullptr, *lat_ml = nullptr;
  char *cq = nullptr, *lq = nullptr, *lat = nullptr, *kv = nullptr, *qabs = nullptr;
  int mixes = 1, lq_ld = 0, cq_ld = 0, kv_ld = 0, max_window = 0, key_cap = 0;  // mixes: blends of h; key_cap: rows of the key workspace
  float *weight = nullptr, *logits = nullptr, *trace_x = nullptr, *sample_scratch = nullptr;
  int *slot_pos = nullptr, *chosen = nullptr, *count = nullptr, *cursor = nullptr, *slot_row = nullptr, *tiles = nullptr, *n_tiles = nullptr, *active = nullptr,
      *active_slot = nullptr, *n_active = nullptr, *next_dev = nullptr;
  float* logits_host = nullptr;     // pinned, LOGIT_ROWS rows
  int* next_host = nullptr;         // pinned
  StepParams *sp_host = nullptr, *sp_dev = nullptr;
  DescBuf big, small;
  int last_rows = 0;
  bool chunk_scan = true;
  int tile = 0;                     // of prompt products (LinArgs::tile)
  ChunkScan scan{};                 // operands of the recurrences over chunks (kernels_chunk_scan.hip)
  int max_chunks = 0;
  float* attn_part = nullptr;       // parts of attention outputs (kernels_mix_few.hip)
  unsigned* attn_arrived = nullptr;
  int splits = 1;                   // attention workgroups per (sequence, key head) of the current decode step: a power of two
  long long fused_layers = 0;       // layers enqueued with the fused decode launches
  std::map<int, Graph> graphs;
  int graph_steps = 0;
  size_t elem() const { return f32 ? 4 : 2; }
};
LayeredModel* lm(dsk_model* m) { return reinterpret_cast<LayeredModel*>(m); }
const LayeredModel* lm(const dsk_model* m) { return reinterpret_cast<const LayeredModel*>(m); }

int dev_alloc(LayeredModel* m, void** p, size_t bytes, bool weight = false) {
  bytes = up(std::max<size_t>(bytes, 16), 256);
  HIP_TRY(hipMalloc(p, bytes));
  m->dev.push_back(*p);
  (weight ? m->weight_bytes : m->scratch_bytes) += (double)bytes;
  HIP_TRY(hipMemsetAsync(*p, 0, bytes, m->ctx->stream));  // padding stays zero for good
  return DSK_OK;
}
template <typename T>
int dev_alloc_n(LayeredModel* m, T** p, size_t n, bool weight = false) {
  return dev_alloc(m, reinterpret_cast<void**>(p), n * sizeof(T), weight);
}

// ---- weights -----------------------------------------------------------------------------------------
// A source hands out a tensor as row-major bf16 in a device scratch buffer (stream order: the next call may overwrite it).
struct Weights {
  LayeredModel* m;
  Checkpoint* ck;       // nullptr: random values
  uint64_t seed = 1;
  uint16_t* raw = nullptr;
  size_t raw_cap = 0;
  ~Weights() {
    if (raw) {
      hipStreamSynchronize(m->ctx->stream);
      hipFree(raw);
    }
  }
  const FileTensor* find(const std::string& name) const {
    auto it = ck->tensors.find(name);
    return it == ck->tensors.end() ? nullptr : &it->second;
  }
  // rows of a matrix whose configuration does not say (dflt: random weights)
  int rows_of(const std::string& name, int dflt, int* out) {
    *out = dflt;
    if (!ck) return DSK_OK;
    const FileTensor* t = find(name);
    if (!t || t->ndim != 2) DSK_FAIL(DSK_ERR_INVALID, "loader: matrix %s is missing", name.c_str());
    *out = t->shape[0];
    return DSK_OK;
  }
  int get(const std::string& name, int rows, int cols, uint16_t** out) {  // rows = 0: a vector
    const size_t n = (size_t)std::max(rows, 1) * cols;
    if (raw_cap < n) {
      HIP_TRY(hipStreamSynchronize(m->ctx->stream));
      if (raw) HIP_TRY(hipFree(raw));
      raw = nullptr;
      raw_cap = 0;
      HIP_TRY(hipMalloc((void**)&raw, n * 2));
      raw_cap = n;
    }
    *out = raw;
    if (!ck) return launch_fill_random(m->ctx->stream, raw, n, rows ? sqrtf(3.f / cols) : 0.1f, seed++);
    const FileTensor* t = find(name);
    if (!t) DSK_FAIL(DSK_ERR_INVALID, "loader: tensor %s is missing", name.c_str());
    const bool ok = rows ? t->ndim == 2 && t->shape[0] == rows && t->shape[1] == cols : t->ndim == 1 && t->shape[0] == cols;
    if (!ok) DSK_FAIL(DSK_ERR_INVALID, "loader: tensor %s has shape [%d, %d], expected [%d, %d]", name.c_str(), t->shape[0], t->shape[1], rows, cols);
    if (t->dtype != "BF16") DSK_FAIL(DSK_ERR_UNSUPPORTED, "loader: tensor %s is %s, expected BF16", name.c_str(), t->dtype.c_str());
    HostSrc src;
    src.fd = ck->fds[t->file];
    src.off = t->off;
    return stage_copy(m->ctx, src, 0, raw, n * 2);
  }
  // a vector (or small table) as 32-bit floats
  int floats(const std::string& name, int rows, int cols, float** out) {
    if (!*out) DSK_TRY(dev_alloc_n(m, out, (size_t)std::max(rows, 1) * cols, true));
    return floats_at(name, rows, cols, *out);
  }
  int floats_at(const std::string& name, int rows, int cols, float* dst) {
    uint16_t* p;
    DSK_TRY(get(name, rows, cols, &p));
    return launch_widen(m->ctx->stream, p, dst, (size_t)std::max(rows, 1) * cols);
  }
  int alloc(PackedMat* p, int rows, int k) {
    p->rows = rows;
    p->k = k;
    p->rt = (int)up(rows, 16) / 16;
    p->kt = (int)up(k, 64) / 32;
    return dev_alloc_n(m, &p->w, p->elems(), true);
  }
  int pack(const std::string& name, int rows, int k, const PackedMat& dst, int row0, int col0 = 0) {
    uint16_t* p;
    DSK_TRY(get(name, rows, k, &p));
    return launch_pack(m->ctx->stream, p, rows, k, dst.w, dst.kt, row0, col0, -1);
  }
  // heads of `rows` rows behind each other, head i's at dst row row0 + i * stride, from row `first` of its `all` rows on; transpose: the
  // head's columns become rows
  int pack_heads(const std::string& name, int heads, int all, int first, int rows, int k, const PackedMat& dst, int row0, int stride, bool transpose = false) {
    uint16_t* p;
    DSK_TRY(get(name, heads * all, k, &p));
    for (int i = 0; i < heads; ++i)
      DSK_TRY(launch_pack(m->ctx->stream, p + ((size_t)i * all + first) * k, rows, k, dst.w, dst.kt, row0 + i * stride, 0, -1, transpose));
    return DSK_OK;
  }
  int matrix(const std::string& name, int rows, int k, PackedMat* dst) {
    DSK_TRY(alloc(dst, rows, k));
    return pack(name, rows, k, *dst, 0);
  }
};

// columns of the shared projection, filled segment by segment: every segment starts at a multiple of `step`
struct Columns {
  struct Part {
    std::string name;
    int rows, col;
  };
  std::vector<Part> parts;
  int next = 0;
  int add(const std::string& name, int rows, int step) {
    next = (int)up(next, step);
    parts.push_back({name, rows, next});
    const int c = next;
    next += rows;
    return c;
  }
};

int load_experts(Weights& W, LayeredModel* m, const MoeSpec& e, LayerW& w) {
  const int D = m->s.width;
  auto one = [&](const std::string& pre, int ff, uint16_t* up_w, uint16_t* down_w, int up_kt, int down_kt) -> int {
    uint16_t* p;
    DSK_TRY(W.get(pre + ".gate", ff, D, &p));
    DSK_TRY(launch_pack(m->ctx->stream, p, ff, D, up_w, up_kt, 0, 0, 0));
    DSK_TRY(W.get(pre + ".up", ff, D, &p));
    DSK_TRY(launch_pack(m->ctx->stream, p, ff, D, up_w, up_kt, 0, 0, 1));
    DSK_TRY(W.get(pre + ".down", D, ff, &p));
    return launch_pack(m->ctx->stream, p, D, ff, down_w, down_kt, 0, 0, -1);
  };
  const int kt = (int)up(D, 64) / 32, drt = (int)up(D, 16) / 16;
  const int urt = (int)up(e.ff, 16) / 8, dkt = (int)up(e.ff, 64) / 32;
  const size_t us = (size_t)urt * kt * 512, ds = (size_t)drt * dkt * 512;
  uint16_t *uw, *dw;
  DSK_TRY(dev_alloc_n(m, &uw, us * e.experts, true));
  DSK_TRY(dev_alloc_n(m, &dw, ds * e.experts, true));
  for (int i = 0; i < e.experts; ++i) DSK_TRY(one(e.name + ".e" + std::to_string(i), e.ff, uw + us * i, dw + ds * i, kt, dkt));
  w.e_up = {uw, nullptr, us, kt, urt, 0, 0};
  w.e_down = {dw, nullptr, ds, dkt, drt, 0, 0};
  if (e.shared_ff) {
    const int surt = (int)up(e.shared_ff, 16) / 8, sdkt = (int)up(e.shared_ff, 64) / 32;
    uint16_t *su, *sd;
    DSK_TRY(dev_alloc_n(m, &su, (size_t)surt * kt * 512, true));
    DSK_TRY(dev_alloc_n(m, &sd, (size_t)drt * sdkt * 512, true));
    DSK_TRY(one(e.name + ".shared", e.shared_ff, su, sd, kt, sdkt));
    w.e_up.shared = su;
    w.e_up.shared_kt = kt;
    w.e_up.shared_rt = surt;
    w.e_down.shared = sd;
    w.e_down.shared_kt = sdkt;
    w.e_down.shared_rt = drt;
  }
  return DSK_OK;
}

int load_layer(Weights& W, LayeredModel* m, const LayerSpec& l, LayerW& w) {
  const int D = m->s.width;
  DSK_TRY(W.floats(l.norm, 0, D, &w.norm));
  Columns wide, narrow;
  int &low_a = w.low_a, &low_g = w.low_g;
  if (l.has_attn) {
    const AttnSpec& a = l.attn;
    w.a_q = wide.add(a.name + ".q", a.heads * a.dim, 16);
    w.a_k = wide.add(a.name + ".k", a.kv_heads * a.dim, 16);
    w.a_v = wide.add(a.name + ".v", a.kv_heads * a.vdim, 16);
  }
  if (l.has_mlstm) {
    const MlstmSpec& a = l.mlstm;
    w.m_q = wide.add(a.name + ".q", a.heads * a.dim, 16);
    w.m_k = wide.add(a.name + ".k", a.heads * a.dim, 16);
    w.m_v = wide.add(a.name + ".v", a.heads * a.vdim, 16);
    w.m_g = wide.add(a.name + ".g", a.heads * a.vdim, 16);
    w.m_i = narrow.add(a.name + ".i", a.heads, 1);
    w.m_f = narrow.add(a.name + ".f", a.heads, 1);
  }
  if (l.has_delta) {
    const DeltaSpec& a = l.delta;
    w.d_q = wide.add(a.name + ".q", a.kv_heads * a.dim, 16);
    w.d_k = wide.add(a.name + ".k", a.kv_heads * a.dim, 16);
    w.d_v = wide.add(a.name + ".v", a.heads * a.vdim, 16);
    if (a.head_decay) {
      w.d_a = narrow.add(a.name + ".a", a.heads, 1);
    } else {
      DSK_TRY(W.rows_of(a.name + ".a1", a.dim, &low_a));
      w.d_low = wide.add(a.name + ".a1", low_a, 64);  // both, behind each other, are one operand of the second product
    }
    if (a.silu_gate) {
      w.d_g = wide.add(a.name + ".g", a.heads * a.vdim, 16);
    } else {
      DSK_TRY(W.rows_of(a.name + ".g1", a.dim, &low_g));
      wide.add(a.name + ".g1", low_g, 1);
    }
    w.d_b = narrow.add(a.name + ".b", a.heads, 1);
  }
  if (l.has_wkv) {
    const WkvSpec& a = l.wkv;
    const int n = a.heads * a.dim;
    w.seg = (int)up(n, 128);  // every projection reads a blend of its own: one operand per `seg` features
    w.w_r = wide.add(a.name + ".r", n, w.seg);
    w.w_k = wide.add(a.name + ".k", n, w.seg);
    w.w_v = wide.add(a.name + ".v", n, w.seg);
    w.w_g = wide.add(a.name + ".g", n, w.seg);
    wide.next = 4 * w.seg;
    DSK_TRY(W.rows_of(a.name + ".w1", std::min(64, a.dim), &low_a));
    w.w_low = narrow.add(a.name + ".w1", low_a, 1);
    narrow.next = (int)up(low_a, 64);  // (an operand of the second product as it is)
  }
  if (l.has_latent) {
    const LatentSpec& a = l.latent;
    w.l_q = narrow.add(a.name + ".dq", a.q_rank, 1);
    w.l_kv = narrow.add(a.name + ".dkv", a.kv_rank + a.rot_dim, 1);
  }
  if (l.has_moe) w.router = narrow.add(l.moe.name + ".router", l.moe.experts, 1);
  w.n_wide = (int)up(wide.next, 64);
  DSK_TRY(W.alloc(&w.proj, w.n_wide + narrow.next, D));
  for (auto& p : wide.parts) DSK_TRY(W.pack(p.name, p.rows, D, w.proj, p.col));
  for (auto& p : narrow.parts) DSK_TRY(W.pack(p.name, p.rows, D, w.proj, w.n_wide + p.col));
  if (l.has_attn || l.has_latent) {
    std::vector<float> f;
    rot_frequencies(l.has_attn ? l.attn.rot : l.latent.rot, &f, &w.rot_amp);
    DSK_TRY(dev_alloc_n(m, &w.freq, f.size(), true));
    HIP_TRY(hipStreamSynchronize(m->ctx->stream));
    if (!f.empty()) HIP_TRY(hipMemcpy(w.freq, f.data(), f.size() * 4, hipMemcpyHostToDevice));
  }
  if (l.has_attn) {
    const AttnSpec& a = l.attn;
    DSK_TRY(W.matrix(a.name + ".o", D, a.heads * a.vdim, &w.a_o));
  }
  if (l.has_mlstm) {
    const MlstmSpec& a = l.mlstm;
    DSK_TRY(W.floats(a.name + ".i.b", 0, a.heads, &w.m_bi));
    DSK_TRY(W.floats(a.name + ".f.b", 0, a.heads, &w.m_bf));
    DSK_TRY(W.floats(a.name + ".norm", 0, a.heads * a.vdim, &w.m_norm));
    DSK_TRY(W.matrix(a.name + ".o", D, a.heads * a.vdim, &w.m_o));
  }
  if (l.has_delta) {
    const DeltaSpec& a = l.delta;
    const int nq = a.kv_heads * a.dim, nv = a.heads * a.vdim;
    DSK_TRY(dev_alloc_n(m, &w.d_conv, (size_t)(2 * nq + nv) * a.taps, true));
    DSK_TRY(W.floats_at(a.name + ".q.conv", nq, a.taps, w.d_conv));
    DSK_TRY(W.floats_at(a.name + ".k.conv", nq, a.taps, w.d_conv + (size_t)nq * a.taps));
    DSK_TRY(W.floats_at(a.name + ".v.conv", nv, a.taps, w.d_conv + (size_t)2 * nq * a.taps));
    DSK_TRY(W.floats(a.name + ".A_log", 0, a.heads, &w.d_rate));  // exp() of it below
    DSK_TRY(launch_exp(m->ctx->stream, w.d_rate, a.heads));
    DSK_TRY(W.floats(a.name + ".dt_bias", 0, a.head_decay ? a.heads : a.heads * a.dim, &w.d_dt));
    DSK_TRY(W.floats(a.name + ".norm", 0, a.vdim, &w.d_norm));
    if (!a.head_decay) {
      DSK_TRY(W.alloc(&w.d_low2, a.heads * (a.dim + a.vdim), low_a + low_g));
      DSK_TRY(W.pack(a.name + ".a2", a.heads * a.dim, low_a, w.d_low2, 0, 0));
      DSK_TRY(W.pack(a.name + ".g2", a.heads * a.vdim, low_g, w.d_low2, a.heads * a.dim, low_a));
    }
    DSK_TRY(W.matrix(a.name + ".o", D, nv, &w.d_o));
  }
  if (l.has_wkv) {
    const WkvSpec& a = l.wkv;
    const int n = a.heads * a.dim;
    DSK_TRY(W.matrix(a.name + ".w2", n, low_a, &w.w_low2));
    DSK_TRY(W.floats(a.name + ".w0", 0, n, &w.w_w0));
    DSK_TRY(W.floats(a.name + ".u", a.heads, a.dim, &w.w_u));
    DSK_TRY(W.floats(a.name + ".norm", 0, n, &w.w_norm));
    DSK_TRY(W.matrix(a.name + ".o", D, n, &w.w_o));
    const char* blends[] = {"r", "k", "v", "g", "w"};  // (as the columns of the projection)
    w.conv.n_mix = 5;
    DSK_TRY(dev_alloc_n(m, &w.conv.mu, 5 * (size_t)D, true));
    for (int i = 0; i < 5; ++i) DSK_TRY(W.floats_at(a.name + ".mu." + blends[i], 0, D, w.conv.mu + (size_t)i * D));
  }
  if (l.has_latent) {
    const LatentSpec& a = l.latent;
    w.dim_p = (int)up(a.dim, 32);
    w.rot_p = (int)up(a.rot_dim, 32);
    w.vdim_p = (int)up(a.vdim, 32);
    w.rank_p = (int)up(a.kv_rank, 64);
    DSK_TRY(W.floats(a.name + ".dq.norm", 0, a.q_rank, &w.l_qn));
    DSK_TRY(W.floats(a.name + ".dkv.norm", 0, a.kv_rank, &w.l_kvn));
    const int hd = w.dim_p + w.rot_p;
    DSK_TRY(W.alloc(&w.l_uq, a.heads * hd, a.q_rank));
    DSK_TRY(W.pack_heads(a.name + ".uq", a.heads, a.dim + a.rot_dim, 0, a.dim, a.q_rank, w.l_uq, 0, hd));
    DSK_TRY(W.pack_heads(a.name + ".uq", a.heads, a.dim + a.rot_dim, a.dim, a.rot_dim, a.q_rank, w.l_uq, w.dim_p, hd));
    DSK_TRY(W.alloc(&w.l_ukv, a.heads * (w.dim_p + w.vdim_p), a.kv_rank));
    DSK_TRY(W.pack_heads(a.name + ".uk", a.heads, a.dim, 0, a.dim, a.kv_rank, w.l_ukv, 0, w.dim_p));
    DSK_TRY(W.alloc(&w.l_abs, a.heads * w.rank_p, a.dim));
    DSK_TRY(W.pack_heads(a.name + ".uk", a.heads, a.dim, 0, a.dim, a.kv_rank, w.l_abs, 0, w.rank_p, true));
    DSK_TRY(W.pack_heads(a.name + ".uv", a.heads, a.vdim, 0, a.vdim, a.kv_rank, w.l_ukv, a.heads * w.dim_p, w.vdim_p));
    DSK_TRY(W.matrix(a.name + ".o", D, a.heads * a.vdim, &w.l_o));
  }
  if (l.sandwich) {
    DSK_TRY(W.floats(l.post, 0, D, &w.post));
    DSK_TRY(W.floats(l.conv, D, l.taps, &w.conv.w));
  }
  if (l.has_dense) {
    const DenseSpec& a = l.dense;
    DSK_TRY(W.floats(l.ff_norm, 0, D, &w.ff_norm));
    DSK_TRY(W.floats(l.ff_post, 0, D, &w.ff_post));
    DSK_TRY(W.floats(l.ff_conv, D, l.taps, &w.ff_conv.w));
    DSK_TRY(W.matrix(a.name + ".up", a.ff, D, &w.ff_up));
    DSK_TRY(W.matrix(a.name + ".down", D, a.ff, &w.ff_down));
    float *act = nullptr, pq[2];
    DSK_TRY(W.floats(a.name + ".act", 0, 2, &act));
    HIP_TRY(hipMemcpyAsync(pq, act, sizeof pq, hipMemcpyDeviceToHost, m->ctx->stream));
    HIP_TRY(hipStreamSynchronize(m->ctx->stream));
    auto softplus = [](double v) { return std::max(v, 0.0) + log1p(exp(-fabs(v))); };
    w.ff_pos = (float)softplus(pq[0]);
    w.ff_neg = (float)(0.5 + softplus(pq[1]));
  }
  if (!l.pair_a.empty()) {
    DSK_TRY(W.floats(l.pair_a, 0, D, &w.pair_a));
    DSK_TRY(W.floats(l.pair_b, 0, D, &w.pair_b));
  }
  if (l.has_moe) DSK_TRY(load_experts(W, m, l.moe, w));
  return DSK_OK;
}

// ---- state layout and workspaces -----------------------------------------------------------------------
void layout_state(LayeredModel* m) {
  size_t off = 0;
  auto take = [&](size_t bytes) {
    const size_t o = off;
    off = up(off + bytes, 256);
    return o;
  };
  for (size_t i = 0; i < m->L.size(); ++i) {
    const LayerSpec& l = m->s.layers[i];
    LayerW& w = m->L[i];
    if (l.has_attn) {
      w.off_k = take((size_t)l.attn.chunk * l.attn.kv_heads * up(l.attn.dim, 32) * m->elem());
      w.off_v = take((size_t)l.attn.chunk * l.attn.kv_heads * up(l.attn.vdim, 32) * m->elem());
    }
    if (l.has_mlstm) {
      w.off_ms = take((size_t)l.mlstm.heads * l.mlstm.dim * l.mlstm.vdim * 4);
      w.off_mn = take((size_t)2 * l.mlstm.heads * l.mlstm.dim * 4);
      w.off_mm = take((size_t)2 * l.mlstm.heads * 4);
    }
    if (l.has_delta) {
      const DeltaSpec& a = l.delta;
      w.off_ds = take((size_t)a.heads * a.dim * a.vdim * 4);
      w.off_dc = take((size_t)2 * (a.taps - 1) * (2 * a.kv_heads * a.dim + a.heads * a.vdim) * 4);
    }
    if (l.has_wkv) {
      w.off_ws = take((size_t)l.wkv.heads * l.wkv.dim * l.wkv.dim * 4);
      w.conv.off_prev = take((size_t)2 * m->s.width * 4);
    }
    if (l.has_latent) w.off_lc = take((size_t)l.latent.window * (w.rank_p + w.rot_p) * m->elem());
    if (l.sandwich) w.conv.off_in = take((size_t)2 * (l.taps - 1) * m->s.width * 4);
    if (l.has_dense) w.ff_conv.off_in = take((size_t)2 * (l.taps - 1) * m->s.width * 4);
  }
  m->seq_bytes = std::max<size_t>(off, 256);
}

int alloc_desc(LayeredModel* m, DescBuf* d, int cap) {
  d->cap = cap;
  size_t off = up(sizeof(SeqDesc) * cap, 16);
  auto take = [&](size_t n) {
    const size_t o = off;
    off += up(n * 4, 16);
    return o;
  };
  d->o_tok = take(cap);
  d->o_row = take(cap);
  d->o_want = take(cap);
  d->o_tile = take(2 * (size_t)cap);
  d->o_chunk = take(2 * (size_t)cap);
  d->o_single = take(cap);
  d->bytes = off;
  HIP_TRY(hipHostMalloc((void**)&d->host, off, hipHostMallocDefault));
  memset(d->host, 0, off);
  return dev_alloc(m, (void**)&d->dev, off);
}

int latent_splits(const LayeredModel* m, const LatentSpec& a) {  // workgroups for a full window
  return (a.window + latent_keys(m->f32) - 1) / latent_keys(m->f32);
}

int alloc_work(LayeredModel* m) {
  const LayeredSpec& s = m->s;
  const size_t n = m->piece, e = m->elem();
  const int D = s.width;
  int low = 0, out = 0, experts = 0, tmax = 1;
  size_t hidden = 0, turn = 0, cq = 0, key = 0, kv = 0, qabs = 0, lat_part = 0, lat_ml = 0;  // (hidden: elements of a row of experts' or dense outputs)
  bool sandwich = false;
  size_t chunk = 0, gates = 0, part = 0, arrived = 0, aq = 0, ak = 0, av = 0, dq = 0, dv = 0, dg = 0, db = 0, o = 0;
  for (size_t i = 0; i < m->L.size(); ++i) {
    const LayerSpec& l = s.layers[i];
    const LayerW& w = m->L[i];
    m->ldw = std::max(m->ldw, w.n_wide);
    m->ldf = std::max(m->ldf, w.proj.rt * 16 - w.n_wide);
    if (l.has_attn) {
      aq = std::max(aq, (size_t)l.attn.heads * up(l.attn.dim, 32));
      ak = std::max(ak, (size_t)l.attn.kv_heads * up(l.attn.dim, 32));
      av = std::max(av, (size_t)l.attn.kv_heads * up(l.attn.vdim, 32));
      out = std::max(out, w.a_o.kt * 32);
      part = std::max(part, (size_t)FEW * l.attn.heads * up(l.attn.chunk, ATTN_SPLIT_KEYS) / ATTN_SPLIT_KEYS * (up(l.attn.vdim, 32) + 2));
      arrived = std::max(arrived, (size_t)FEW * l.attn.kv_heads);
    }
    if (l.has_mlstm) {
      o = std::max(o, (size_t)l.mlstm.heads * (l.mlstm.vdim + 1));
      chunk = std::max(chunk, l.mlstm.heads * chunk_floats(l.mlstm.dim));
      gates = std::max(gates, (size_t)l.mlstm.heads);
      out = std::max(out, w.m_o.kt * 32);
    }
    if (l.has_delta) {
      const DeltaSpec& a = l.delta;
      dq = std::max(dq, (size_t)a.kv_heads * a.dim);
      dg = std::max(dg, (size_t)a.heads * a.dim);
      dv = std::max(dv, (size_t)a.heads * a.vdim);
      db = std::max(db, (size_t)a.heads);
      chunk = std::max(chunk, a.heads * chunk_floats(a.dim));
      o = std::max(o, (size_t)a.heads * a.vdim);
      low = std::max(low, w.d_low2.rt * 16);
      out = std::max(out, w.d_o.kt * 32);
    }
    if (l.has_wkv) {
      const WkvSpec& a = l.wkv;
      m->mixes = std::max(m->mixes, w.conv.n_mix);
      chunk = std::max(chunk, a.heads * chunk_floats(a.dim));
      o = std::max(o, (size_t)a.heads * a.dim);
      low = std::max(low, w.w_low2.rt * 16);
      out = std::max(out, w.w_o.kt * 32);
    }
    if (l.has_latent) {
      const LatentSpec& a = l.latent;
      m->max_window = std::max(m->max_window, a.window);
      cq = std::max(cq, (size_t)w.l_uq.kt * 32);
      turn = std::max(turn, (size_t)a.rot.dims);
      m->lq_ld = std::max(m->lq_ld, w.l_uq.rt * 16 + 64);  // (the last head's columns, read in groups of 64)
      key = std::max(key, (size_t)w.rank_p + w.rot_p);
      kv = std::max(kv, (size_t)w.l_ukv.rt * 16);
      qabs = std::max(qabs, (size_t)a.heads * w.rank_p);
      lat_part = std::max(lat_part, (size_t)FEW * a.heads * latent_splits(m, a) * w.rank_p);
      lat_ml = std::max(lat_ml, (size_t)FEW * a.heads * latent_splits(m, a) * 2);
      out = std::max(out, w.l_o.kt * 32);
    }
    sandwich |= l.sandwich;
    if (l.has_dense) {
      m->hid_ld = std::max(m->hid_ld, w.ff_down.kt * 32);
      hidden = std::max<size_t>(hidden, 1);
    }
    if (l.has_moe) {
      const MoeSpec& q = l.moe;
      experts = std::max(experts, q.experts);
      tmax = std::max(tmax, q.top + (q.shared_ff > 0));
      hidden = std::max<size_t>(hidden, q.top + (q.shared_ff > 0));
      m->hid_ld = std::max({m->hid_ld, w.e_down.kt * 32, w.e_down.shared_kt * 32});
    }
  }
  m->h_ld = (int)up(D, 64);
  m->mix_ld = m->y_ld = (int)up(D, 16);
  m->out_ld = std::max(out, 64);
  m->cq_ld = (int)cq;
  m->kv_ld = (int)kv;
  m->low_ld = low;
  m->slots = tmax;
  m->ld_logits = m->head.rt * 16;
  DSK_TRY(dev_alloc_n(m, &m->x, n * D));
  DSK_TRY(dev_alloc(m, (void**)&m->h, n * m->h_ld * e * m->mixes));
  if (sandwich) DSK_TRY(dev_alloc_n(m, &m->h_f, n * D));
  if (m->max_window) {
    m->key_cap = m->piece + m->max_window;
    DSK_TRY(dev_alloc_n(m, &m->turn, n * turn));
    DSK_TRY(dev_alloc(m, (void**)&m->cq, n * m->cq_ld * e));
    DSK_TRY(dev_alloc(m, (void**)&m->lq, n * m->lq_ld * e));
    DSK_TRY(dev_alloc(m, (void**)&m->lat, m->key_cap * key * e));
    DSK_TRY(dev_alloc(m, (void**)&m->kv, m->key_cap * m->kv_ld * e));
    DSK_TRY(dev_alloc(m, (void**)&m->qabs, FEW * qabs * e));
    DSK_TRY(dev_alloc_n(m, &m->lat_part, lat_part));
    DSK_TRY(dev_alloc_n(m, &m->lat_ml, lat_ml));
  }
  DSK_TRY(dev_alloc(m, (void**)&m->hw, n * m->h_ld * e));
  DSK_TRY(dev_alloc(m, (void**)&m->wide, n * m->ldw * e));
  DSK_TRY(dev_alloc_n(m, &m->narrow, n * m->ldf));
  DSK_TRY(dev_alloc(m, (void**)&m->out_a, n * m->out_ld * e));
  DSK_TRY(dev_alloc(m, (void**)&m->out_b, n * m->out_ld * e));
  const size_t mix_rows = std::max<size_t>(n * MIX_PARTS, FEW * MIX_PARTS_FEW);
  DSK_TRY(dev_alloc_n(m, &m->mix_a, mix_rows * m->mix_ld));
  DSK_TRY(dev_alloc_n(m, &m->mix_b, mix_rows * m->mix_ld));
  DSK_TRY(dev_alloc(m, (void**)&m->qb, n * aq * e));
  DSK_TRY(dev_alloc(m, (void**)&m->kb, n * ak * e));
  DSK_TRY(dev_alloc(m, (void**)&m->vb, n * av * e));
  DSK_TRY(dev_alloc_n(m, &m->low, n * low));
  DSK_TRY(dev_alloc_n(m, &m->dq, n * dq));
  DSK_TRY(dev_alloc_n(m, &m->dk, n * dq));
  DSK_TRY(dev_alloc_n(m, &m->dv, n * dv));
  DSK_TRY(dev_alloc_n(m, &m->dg, n * dg));
  DSK_TRY(dev_alloc_n(m, &m->db, n * db));
  DSK_TRY(dev_alloc_n(m, &m->o, n * o));
  if (m->chunk_scan && chunk) {
    m->max_chunks = m->piece / RECUR_CHUNK + 32;
    DSK_TRY(dev_alloc_n(m, &m->scan.ops, m->max_chunks * chunk));
    DSK_TRY(dev_alloc_n(m, &m->scan.keep, n * gates));
    DSK_TRY(dev_alloc_n(m, &m->scan.add, n * gates));
    DSK_TRY(dev_alloc_n(m, &m->scan.floor, n * gates));
  }
  DSK_TRY(dev_alloc_n(m, &m->attn_part, part));
  DSK_TRY(dev_alloc_n(m, &m->attn_arrived, arrived));
  if (hidden) DSK_TRY(dev_alloc(m, (void**)&m->hidden, n * hidden * m->hid_ld * e));
  if (experts) {
    const size_t ns = n * tmax;
    m->max_tiles = (int)(ns / MOE_TILE) + experts + 2;
    DSK_TRY(dev_alloc(m, (void**)&m->y, ns * m->y_ld * e));
    DSK_TRY(dev_alloc_n(m, &m->weight, ns));
    DSK_TRY(dev_alloc_n(m, &m->slot_pos, ns));
    DSK_TRY(dev_alloc_n(m, &m->chosen, ns));
    DSK_TRY(dev_alloc_n(m, &m->slot_row, ns));
    DSK_TRY(dev_alloc_n(m, &m->count, experts));
    DSK_TRY(dev_alloc_n(m, &m->cursor, experts));
    DSK_TRY(dev_alloc_n(m, &m->tiles, 4 * (size_t)m->max_tiles));
    DSK_TRY(dev_alloc_n(m, &m->n_tiles, 1));
    DSK_TRY(dev_alloc_n(m, &m->active, experts + 1));
    DSK_TRY(dev_alloc_n(m, &m->active_slot, (size_t)(experts + 1) * FEW));
    DSK_TRY(dev_alloc_n(m, &m->n_active, 1));
  }
  DSK_TRY(dev_alloc_n(m, &m->logits, (size_t)LOGIT_ROWS * m->ld_logits));
  DSK_TRY(dev_alloc_n(m, &m->next_dev, LOGIT_ROWS));
  DSK_TRY(dev_alloc(m, (void**)&m->sample_scratch, FEW * sample_scratch_bytes()));
  DSK_TRY(dev_alloc_n(m, &m->sp_dev, FEW));
  HIP_TRY(hipHostMalloc((void**)&m->sp_host, sizeof(StepParams) * FEW, hipHostMallocDefault));
  memset(m->sp_host, 0, sizeof(StepParams) * FEW);
  HIP_TRY(hipHostMalloc((void**)&m->logits_host, (size_t)LOGIT_ROWS * s.vocab * 4, hipHostMallocDefault));
  HIP_TRY(hipHostMalloc((void**)&m->next_host, LOGIT_ROWS * 4, hipHostMallocDefault));
  DSK_TRY(alloc_desc(m, &m->big, m->piece));
  DSK_TRY(alloc_desc(m, &m->small, FEW));
  return DSK_OK;
}

// ---- one pass --------------------------------------------------------------------------------------------
LinArgs lin(const PackedMat& w, const void* a, int lda, int rows) {
  LinArgs l{};
  l.w = w.w;
  l.a_t = a;
  l.lda = lda;
  l.kt = w.kt;
  l.rt = w.rt;
  l.rows = rows;
  return l;
}
LinArgs lin_f(const PackedMat& w, const void* a, int lda, int rows, float* out, int ld) {  // 32-bit output
  LinArgs l = lin(w, a, lda, rows);
  l.out_f = out;
  l.ld_f = ld;
  return l;
}
// A product whose output the next residual sum reads (mix_a; second: mix_b), split over k where its tiles alone leave compute units idle
LinArgs mix_lin(LayeredModel* m, const PackedMat& w, const void* a, int lda, int rows, bool few, bool second = false) {
  LinArgs l = lin_f(w, a, lda, rows, second ? m->mix_b : m->mix_a, m->mix_ld);
  l.parts = m->mix_parts[second] = few ? lin_parts_few(w.rt, w.kt, MIX_PARTS_FEW) : lin_parts(rows, w.rt, w.kt, m->f32, MIX_PARTS);
  l.part_stride = m->mix_stride = (size_t)rows * m->mix_ld;
  return l;
}
int run_lin(LayeredModel* m, const LinArgs* a, int n, bool few) {
  if (few) return launch_lin_few(m->ctx->stream, a, n, m->f32);
  for (int i = 0; i < n; ++i) {
    LinArgs l = a[i];
    l.tile = m->tile;
    DSK_TRY(launch_lin(m->ctx->stream, l, m->f32));
  }
  return DSK_OK;
}

// the residual sum in front of layer l (l = layers: behind the last one)
JoinArgs join_args(LayeredModel* m, const PassDesc& p, int l) {
  JoinArgs j{};
  j.p = p;
  j.width = m->s.width;
  j.h_ld = m->h_ld;
  j.eps = (float)m->s.eps;
  j.norm_offset = (float)m->s.norm_offset;
  j.x = m->x;
  j.h_t = m->h;
  j.mix_ld = m->mix_ld;
  if (l == 0) {
    j.embed = m->embed;
    return j;
  }
  const LayerSpec& s = m->s.layers[l - 1];
  const LayerW& w = m->L[l - 1];
  j.mix_a = m->mix_a;
  j.parts_a = m->mix_parts[0];
  j.parts_b = m->mix_parts[1];
  j.mix_stride = m->mix_stride;
  j.post_w = s.has_dense ? w.ff_post : w.post;
  if (w.pair_a) {
    j.mix_b = m->mix_b;
    j.pair_wa = w.pair_a;
    j.pair_wb = w.pair_b;
  }
  if (s.has_moe) {
    j.y_t = m->y;
    j.y_ld = m->y_ld;
    j.n_slots = s.moe.top + (s.moe.shared_ff > 0);
    j.slot_pos = m->slot_pos;
    j.weight = m->weight;
  }
  return j;
}

ChunkAttnArgs attn_args(LayeredModel* m, const PassDesc& p, const LayerSpec& l, const LayerW& w) {
  const AttnSpec& s = l.attn;
  ChunkAttnArgs a{};
  a.p = p;
  a.heads = s.heads;
  a.kv_heads = s.kv_heads;
  a.dim = s.dim;
  a.vdim = s.vdim;
  a.dim_p = (int)up(s.dim, 32);
  a.vdim_p = (int)up(s.vdim, 32);
  a.chunk = s.chunk;
  a.scale = (float)s.scale;
  a.eps = (float)m->s.eps;
  a.proj_t = m->wide;
  a.ld = m->ldw;
  a.col_q = w.a_q;
  a.col_k = w.a_k;
  a.col_v = w.a_v;
  a.freq = w.freq;
  a.rot_dims = s.rot.dims;
  a.rot_amp = w.rot_amp;
  a.q_t = m->qb;
  a.k_t = m->kb;
  a.v_t = m->vb;
  a.off_k = w.off_k;
  a.off_v = w.off_v;
  a.out_t = m->out_a;
  a.out_ld = m->out_ld;
  return a;
}
int attention(LayeredModel* m, const ChunkAttnArgs& a) {
  hipStream_t st = m->ctx->stream;
  DSK_TRY(launch_chunk_prep(st, a, m->f32));
  DSK_TRY(launch_chunk_attn(st, a, m->f32));
  return launch_chunk_store(st, a, m->f32);
}
MlstmArgs mlstm_args(LayeredModel* m, const PassDesc& p, const LayerSpec& l, const LayerW& w, char* out) {
  const MlstmSpec& s = l.mlstm;
  MlstmArgs a{};
  a.p = p;
  a.heads = s.heads;
  a.dim = s.dim;
  a.vdim = s.vdim;
  a.q_scale = 1.f / sqrtf((float)s.dim);
  a.gate_cap = (float)s.gate_cap;
  a.floor_eps = (float)s.floor_eps;
  a.eps = (float)m->s.eps;
  a.proj_t = m->wide;
  a.ld = m->ldw;
  a.col_q = w.m_q;
  a.col_k = w.m_k;
  a.col_v = w.m_v;
  a.col_g = w.m_g;
  a.gate_f = m->narrow;
  a.ld_gate = m->ldf;
  a.col_i = w.m_i;
  a.col_f = w.m_f;
  a.b_i = w.m_bi;
  a.b_f = w.m_bf;
  a.out_norm = w.m_norm;
  a.o = m->o;
  a.off_s = w.off_ms;
  a.off_n = w.off_mn;
  a.off_m = w.off_mm;
  a.out_t = out;
  a.out_ld = m->out_ld;
  return a;
}
// a pass of few, long sequences runs its recurrences over chunks of 16 tokens; many short ones go token by token
bool in_chunks(const LayeredModel* m, const PassDesc& p) { return m->chunk_scan && p.n_chunks <= m->max_chunks && p.rows >= 4 * p.n_seqs; }
int mlstm(LayeredModel* m, const MlstmArgs& a) {
  const bool chunks = in_chunks(m, a.p);
  if (chunks) DSK_TRY(launch_mlstm_chunks(m->ctx->stream, a, m->scan, m->f32));
  else DSK_TRY(launch_mlstm_scan(m->ctx->stream, a, m->f32));
  return launch_mlstm_out(m->ctx->stream, a, chunks ? &m->scan : nullptr, m->f32);
}
DeltaArgs delta_args(LayeredModel* m, const PassDesc& p, const LayerSpec& l, const LayerW& w) {
  const DeltaSpec& s = l.delta;
  DeltaArgs a{};
  a.p = p;
  a.heads = s.heads;
  a.kv_heads = s.kv_heads;
  a.dim = s.dim;
  a.vdim = s.vdim;
  a.taps = s.taps;
  a.unit_eps = (float)s.unit_eps;
  a.q_scale = 1.f / sqrtf((float)s.dim);
  a.eps = (float)m->s.eps;
  a.proj_t = m->wide;
  a.ld = m->ldw;
  a.col_q = w.d_q;
  a.col_k = w.d_k;
  a.col_v = w.d_v;
  a.gate_f = m->narrow;
  a.ld_gate = m->ldf;
  a.col_b = w.d_b;
  a.low_f = m->low;
  a.ld_low = m->low_ld;
  a.conv_w = w.d_conv;
  a.a_rate = w.d_rate;
  a.head_decay = s.head_decay;
  a.col_a = w.d_a;
  a.silu_gate = s.silu_gate;
  a.col_g = w.d_g;
  a.dt_bias = w.d_dt;
  a.out_norm = w.d_norm;
  a.q = m->dq;
  a.k = m->dk;
  a.v = m->dv;
  a.g = m->dg;
  a.beta = m->db;
  a.o = m->o;
  a.off_s = w.off_ds;
  a.off_conv = w.off_dc;
  a.out_t = m->out_a;
  a.out_ld = m->out_ld;
  return a;
}
int delta(LayeredModel* m, const DeltaArgs& a, const LayerW& w, bool few) {
  if (!a.head_decay) {
    const LinArgs low = lin_f(w.d_low2, m->wide + (size_t)w.d_low * m->elem(), m->ldw, a.p.rows, m->low, m->low_ld);
    DSK_TRY(run_lin(m, &low, 1, few));
  }
  DSK_TRY(launch_delta_prep(m->ctx->stream, a, m->f32));
  if (in_chunks(m, a.p)) DSK_TRY(launch_delta_chunks(m->ctx->stream, a, m->scan));
  else DSK_TRY(launch_delta_scan(m->ctx->stream, a));
  return launch_delta_out(m->ctx->stream, a, m->f32);
}
MoeArgs moe_args(LayeredModel* m, const PassDesc& p, const LayerSpec& l, const LayerW& w) {
  const MoeSpec& s = l.moe;
  MoeArgs a{};
  a.rows = p.rows;
  a.width_ld = m->h_ld;
  a.experts = s.experts;
  a.top = s.top;
  a.shared = s.shared_ff > 0;
  a.logits = m->narrow + w.router;
  a.ld_logits = m->ldf;
  a.weight = m->weight;
  a.slot_pos = m->slot_pos;
  a.chosen = m->chosen;
  a.count = m->count;
  a.cursor = m->cursor;
  a.slot_row = m->slot_row;
  a.tiles = m->tiles;
  a.n_tiles = m->n_tiles;
  a.max_tiles = std::min(m->max_tiles, p.rows * s.top / MOE_TILE + std::min(s.experts, p.rows * s.top) + (a.shared ? (p.rows + MOE_TILE - 1) / MOE_TILE : 0));
  a.active = m->active;
  a.active_slot = m->active_slot;
  a.n_active = m->n_active;
  a.max_active = std::min(s.experts, p.rows * s.top) + a.shared;
  a.h_t = m->h;
  a.hidden_t = m->hidden;
  a.hidden_ld = m->hid_ld;
  a.y_t = m->y;
  a.y_ld = m->y_ld;
  a.up = w.e_up;
  a.down = w.e_down;
  a.limit = (float)s.limit;
  a.shared_limit = (float)s.shared_limit;
  a.alpha = (float)s.alpha;
  a.offset = (float)s.up_offset;
  return a;
}

WkvArgs wkv_args(LayeredModel* m, const PassDesc& p, const LayerSpec& l, const LayerW& w) {
  WkvArgs a{};
  a.p = p;
  a.heads = l.wkv.heads;
  a.dim = l.wkv.dim;
  a.eps = (float)m->s.eps;
  a.proj_t = m->wide;
  a.ld = m->ldw;
  a.col_r = w.w_r;
  a.col_k = w.w_k;
  a.col_v = w.w_v;
  a.col_g = w.w_g;
  a.low_f = m->low;
  a.ld_low = m->low_ld;
  a.w0 = w.w_w0;
  a.u = w.w_u;
  a.out_norm = w.w_norm;
  a.o = m->o;
  a.off_s = w.off_ws;
  a.out_t = m->out_a;
  a.out_ld = m->out_ld;
  return a;
}
int wkv(LayeredModel* m, const WkvArgs& a, const LayerW& w, bool few) {
  hipStream_t st = m->ctx->stream;
  // the decay's second product multiplies 32-bit activations, in bfloat16 runs too
  const LinArgs low = lin_f(w.w_low2, m->narrow + w.w_low, m->ldf, a.p.rows, m->low, m->low_ld);
  DSK_TRY(few ? launch_lin_few(st, &low, 1, true) : launch_lin(st, low, true));
  if (in_chunks(m, a.p)) DSK_TRY(launch_wkv_chunks(st, a, m->scan, m->f32));
  else DSK_TRY(launch_wkv_scan(st, a, m->f32));
  return launch_wkv_out(st, a, m->f32);
}
LatentArgs latent_args(LayeredModel* m, const PassDesc& p, const LayerSpec& l, const LayerW& w) {
  const LatentSpec& s = l.latent;
  LatentArgs a{};
  a.p = p;
  a.heads = s.heads;
  a.dim = s.dim;
  a.rot_dim = s.rot_dim;
  a.vdim = s.vdim;
  a.q_rank = s.q_rank;
  a.kv_rank = s.kv_rank;
  a.window = s.window;
  a.rot_dims = s.rot.dims;
  a.dim_p = w.dim_p;
  a.rot_p = w.rot_p;
  a.vdim_p = w.vdim_p;
  a.rank_p = w.rank_p;
  a.scale = (float)s.scale;
  a.eps = (float)m->s.eps;
  a.proj_f = m->narrow;
  a.ld = m->ldf;
  a.col_q = w.l_q;
  a.col_kv = w.l_kv;
  a.q_norm = w.l_qn;
  a.kv_norm = w.l_kvn;
  a.freq = w.freq;
  a.cq_t = m->cq;
  a.cq_ld = m->cq_ld;
  a.turn = m->turn;
  a.q_t = m->lq;
  a.q_ld = m->lq_ld;
  a.lat_t = m->lat;
  a.kv_t = m->kv;
  a.kv_ld = m->kv_ld;
  a.off_c = w.off_lc;
  a.out_t = m->out_a;
  a.out_ld = m->out_ld;
  a.splits = std::min(m->splits, latent_splits(m, s));
  a.qa_t = m->qabs;
  a.part = m->lat_part;
  a.part_ml = m->lat_ml;
  a.up_w = w.l_ukv.w;
  a.up_kt = w.l_ukv.kt;
  a.up_row = s.heads * w.dim_p;
  return a;
}
int latent(LayeredModel* m, LatentArgs a, const LayerW& w, bool few) {
  hipStream_t st = m->ctx->stream;
  DSK_TRY(launch_latent_prep(st, a, m->f32));
  auto to_t = [&](LinArgs l, void* out, int ld) {  // everything in the activations' type
    l.n_wide = l.rt * 16;
    l.out_t = out;
    l.ld_t = ld;
    return l;
  };
  const LinArgs uq = to_t(lin(w.l_uq, m->cq, a.cq_ld, a.p.rows), m->lq, m->lq_ld);
  DSK_TRY(run_lin(m, &uq, 1, few));
  if (a.p.key_rows) {
    DSK_TRY(launch_latent_gather(st, a, m->f32));
    const LinArgs ukv = to_t(lin(w.l_ukv, m->lat, w.rank_p + w.rot_p, a.p.key_rows), m->kv, a.kv_ld);
    DSK_TRY(run_lin(m, &ukv, 1, false));
    DSK_TRY(launch_latent_turn(st, a, m->f32));
    DSK_TRY(launch_latent_attn(st, a, m->f32));
    DSK_TRY(launch_latent_store(st, a, m->f32));
  }
  for (a.first = 0; a.first < a.p.n_single; a.first += FEW) {
    a.n = std::min((int)FEW, a.p.n_single - a.first);
    LinArgs qa = to_t(lin(w.l_abs, m->lq, m->lq_ld, a.n), m->qabs, a.heads * w.rank_p);
    qa.a_seg = w.rank_p;  // a head's features read its part of the queries
    qa.a_ops = a.heads;
    qa.a_stride = w.dim_p + w.rot_p;
    if (!few) {
      qa.row_seq = a.p.single + a.first;
      qa.seqs = a.p.seqs;
    }
    DSK_TRY(launch_lin_few(st, &qa, 1, m->f32));
    DSK_TRY(launch_latent_few(st, a, m->f32));
  }
  return DSK_OK;
}

ConvArgs conv_args(LayeredModel* m, const PassDesc& p, const LayerSpec& l, const ConvW& c) {
  ConvArgs a{};
  a.taps = l.taps;
  a.w = c.w;
  a.off_in = c.off_in;
  a.mu = c.mu;
  a.n_mix = c.n_mix;
  a.off_prev = c.off_prev;
  a.out_t = m->h;
  a.ld = m->h_ld;
  a.mix_stride = (size_t)p.rows * m->h_ld;
  return a;
}
// the residual sum and norm in front of a sublayer, and the convolution a sandwich layer has there
int enter(LayeredModel* m, JoinArgs j, const float* norm_w, const LayerSpec& s, const ConvW& c, bool few) {
  j.norm_w = norm_w;
  if (!s.sandwich) return launch_join(m->ctx->stream, j, m->f32);
  const ConvArgs conv = conv_args(m, j.p, s, c);
  if (few && m->fused_decode) {
    j.conv = conv;
    return launch_join(m->ctx->stream, j, m->f32);
  }
  j.h_f = m->h_f;
  DSK_TRY(launch_join(m->ctx->stream, j, m->f32));
  return launch_conv(m->ctx->stream, j.p, m->s.width, m->h_f, conv, m->f32);
}
int run_layer(LayeredModel* m, const PassDesc& p, int l, bool few) {
  const LayerSpec& s = m->s.layers[l];
  const LayerW& w = m->L[l];
  hipStream_t st = m->ctx->stream;
  DSK_TRY(enter(m, join_args(m, p, l), w.norm, s, w.conv, few));
  if (m->trace && l > 0) HIP_TRY(hipMemcpyAsync(m->trace_x + (size_t)(l - 1) * m->piece * m->s.width, m->x, (size_t)p.rows * m->s.width * 4, hipMemcpyDeviceToDevice, st));
  LinArgs pr = lin(w.proj, m->h, m->h_ld, p.rows);
  pr.n_wide = w.n_wide;
  pr.out_t = m->wide;
  pr.ld_t = m->ldw;
  pr.out_f = m->narrow;
  pr.ld_f = m->ldf;
  if (s.has_wkv) {
    pr.epi = LIN_TANH_F;
    pr.a_seg = w.seg;
    pr.a_ops = w.conv.n_mix;
    pr.a_stride = (size_t)p.rows * m->h_ld;
  }
  DSK_TRY(run_lin(m, &pr, 1, few));
  // the mixers' outputs and their products: attention or the only mixer in `a`, the second of a pair in `b`
  LinArgs outs[2];
  int n_out = 0;
  MixFewArgs f{};
  if (s.has_attn) {
    f.attn = attn_args(m, p, s, w);
    outs[n_out++] = mix_lin(m, w.a_o, m->out_a, m->out_ld, p.rows, few);
  }
  if (s.has_mlstm) {
    f.mlstm = mlstm_args(m, p, s, w, n_out ? m->out_b : m->out_a);
    outs[n_out] = mix_lin(m, w.m_o, n_out ? m->out_b : m->out_a, m->out_ld, p.rows, few, n_out > 0);
    ++n_out;
  }
  if (s.has_delta) {
    f.delta = delta_args(m, p, s, w);
    outs[n_out++] = mix_lin(m, w.d_o, m->out_a, m->out_ld, p.rows, few);
  }
  if (s.has_wkv) {
    f.wkv = wkv_args(m, p, s, w);
    outs[n_out++] = mix_lin(m, w.w_o, m->out_a, m->out_ld, p.rows, few);
  }
  if (s.has_latent) outs[n_out++] = mix_lin(m, w.l_o, m->out_a, m->out_ld, p.rows, few);
  const MoeArgs e = s.has_moe ? moe_args(m, p, s, w) : MoeArgs{};
  f.rows = p.rows;
  f.has_attn = s.has_attn;
  f.has_mlstm = s.has_mlstm;
  f.has_delta = s.has_delta;
  f.has_wkv = s.has_wkv;
  f.has_route = s.has_moe;
  f.moe = e;
  f.splits = s.has_attn ? std::min(m->splits, (s.attn.chunk + ATTN_SPLIT_KEYS - 1) / ATTN_SPLIT_KEYS) : 0;
  f.part = m->attn_part;
  f.arrived = m->attn_arrived;
  const PackedMat& low2 = s.has_wkv ? w.w_low2 : w.d_low2;
  f.low_w = low2.w;
  f.low_kt = low2.kt;
  f.low_a = w.low_a;
  f.low_g = w.low_g;
  f.col_low = w.d_low;
  f.wkv_low = m->narrow + w.w_low;
  f.wkv_low_ld = m->ldf;
  const bool fused = few && m->fused_decode && !s.has_latent && mix_few_fits(f);
  if (s.has_latent) DSK_TRY(latent(m, latent_args(m, p, s, w), w, few));
  if (fused) {
    DSK_TRY(launch_mix_few(st, f, m->f32));
    m->fused_layers++;
  } else {
    if (s.has_attn) DSK_TRY(attention(m, f.attn));
    if (s.has_mlstm) DSK_TRY(mlstm(m, f.mlstm));
    if (s.has_delta) DSK_TRY(delta(m, f.delta, w, few));
    if (s.has_wkv) DSK_TRY(wkv(m, f.wkv, w, few));
  }
  if (s.has_dense) {
    DSK_TRY(run_lin(m, outs, n_out, few));
    JoinArgs j = join_args(m, p, l);
    j.embed = nullptr;
    j.y_t = nullptr;
    j.mix_a = m->mix_a;
    j.parts_a = m->mix_parts[0];
    j.mix_stride = m->mix_stride;
    j.mix_b = nullptr;
    j.post_w = w.post;
    DSK_TRY(enter(m, j, w.ff_norm, s, w.ff_conv, few));
    LinArgs u = lin(w.ff_up, m->h, m->h_ld, p.rows);
    u.epi = LIN_XIELU;
    u.p0 = w.ff_pos;
    u.p1 = w.ff_neg;
    u.n_wide = w.ff_up.rt * 16;
    u.out_t = m->hidden;
    u.ld_t = m->hid_ld;
    DSK_TRY(run_lin(m, &u, 1, few));
    const LinArgs d = mix_lin(m, w.ff_down, m->hidden, m->hid_ld, p.rows, few);
    return run_lin(m, &d, 1, few);
  }
  if (!s.has_moe) return run_lin(m, outs, n_out, few);
  if (few) {
    if (!fused) DSK_TRY(launch_route_few(st, e));
    DSK_TRY(launch_experts_few(st, e, false, nullptr, 0, m->f32));
    return launch_experts_few(st, e, true, outs, n_out, m->f32);
  }
  DSK_TRY(run_lin(m, outs, n_out, few));
  DSK_TRY(launch_route(st, e));
  DSK_TRY(launch_experts(st, e, false, m->f32));
  return launch_experts(st, e, true, m->f32);
}

// logits of hw rows [r0, r0 + n) into m->logits
int run_head(LayeredModel* m, int r0, int n) {
  LinArgs a = lin_f(m->head, m->hw + (size_t)r0 * m->h_ld * m->elem(), m->h_ld, n, m->logits, m->ld_logits);
  if (m->s.softcap > 0) {
    a.epi = LIN_SOFTCAP;
    a.p0 = (float)m->s.softcap;
  } else if (m->s.logit_scale != 1.0) {
    a.epi = LIN_SCALE;
    a.p0 = (float)m->s.logit_scale;
  }
  return run_lin(m, &a, 1, n <= FEW);
}
int run_choice(LayeredModel* m, int n, int mode) {  // the next token of every row of m->logits
  hipStream_t st = m->ctx->stream;
  if (mode == OUT_SAMPLE) HIP_TRY(hipMemcpyAsync(m->sp_dev, m->sp_host, sizeof(StepParams) * n, hipMemcpyHostToDevice, st));
  for (int i = 0; i < n; ++i) {
    const float* lg = m->logits + (size_t)i * m->ld_logits;
    if (mode == OUT_ARGMAX) DSK_TRY(launch_argmax(st, lg, m->s.vocab, m->next_dev + i));
    else DSK_TRY(launch_sample(st, lg, m->s.vocab, m->sp_dev + i, 0.f, 0.f, 0.f, m->sample_scratch + (size_t)i * (sample_scratch_bytes() / 4), m->next_dev + i));
  }
  HIP_TRY(hipMemcpyAsync(m->next_host, m->next_dev, (size_t)n * 4, hipMemcpyDeviceToHost, st));
  return DSK_OK;
}

PassDesc pass_desc(const DescBuf& d, int rows, int n_seqs, int n_want, int n_tiles, int n_chunks) {
  PassDesc p{};
  p.seqs = reinterpret_cast<const SeqDesc*>(d.dev);
  p.tokens = reinterpret_cast<const int*>(d.dev + d.o_tok);
  p.row_seq = reinterpret_cast<const int*>(d.dev + d.o_row);
  p.want = reinterpret_cast<const int*>(d.dev + d.o_want);
  p.qtile = reinterpret_cast<const int*>(d.dev + d.o_tile);
  p.chunk = reinterpret_cast<const int*>(d.dev + d.o_chunk);
  p.single = reinterpret_cast<const int*>(d.dev + d.o_single);
  p.rows = rows;
  p.n_seqs = n_seqs;
  p.n_want = n_want;
  p.n_qtiles = n_tiles;
  p.n_chunks = n_chunks;
  return p;
}

// every launch of a pass up to the final norm of the wanted rows (in m->hw)
int run_body(LayeredModel* m, const DescBuf& d, const PassDesc& p, bool few) {
  hipStream_t st = m->ctx->stream;
  const int n = (int)m->L.size();
  HIP_TRY(hipMemcpyAsync(d.dev, d.host, d.bytes, hipMemcpyHostToDevice, st));
  for (int l = 0; l < n; ++l) DSK_TRY(run_layer(m, p, l, few));
  JoinArgs j = join_args(m, p, n);
  if (m->trace) {
    DSK_TRY(launch_join(st, j, m->f32));
    HIP_TRY(hipMemcpyAsync(m->trace_x + (size_t)(n - 1) * m->piece * m->s.width, m->x, (size_t)p.rows * m->s.width * 4, hipMemcpyDeviceToDevice, st));
    j.mix_a = j.mix_b = nullptr;
    j.y_t = nullptr;
  }
  if (p.n_want == 0) return DSK_OK;
  j.norm_w = m->final_norm;
  j.h_t = m->hw;
  j.only_want = 1;
  return launch_join(st, j, m->f32);
}
int run_few(LayeredModel* m, const PassDesc& p, int mode) {
  DSK_TRY(run_body(m, m->small, p, true));
  if (p.n_want == 0) return DSK_OK;
  DSK_TRY(run_head(m, 0, p.n_want));
  if (mode == OUT_ARGMAX || mode == OUT_SAMPLE) return run_choice(m, p.n_want, mode);
  HIP_TRY(hipMemcpy2DAsync(m->logits_host, (size_t)m->s.vocab * 4, m->logits, (size_t)m->ld_logits * 4, (size_t)m->s.vocab * 4, p.n_want, hipMemcpyDeviceToHost, m->ctx->stream));
  return DSK_OK;
}

// keys in front of a portion that starts at `pos` which a window of the model may reach
int older_keys(const LayeredModel* m, int pos) { return m->max_window ? std::min(pos, m->max_window - 1) : 0; }

struct Part {   // a portion of one entry inside a pass
  int entry, first, len;
};
// One pass over `parts`; wanted rows come from `want` (rows of the pass).  out: logits of the wanted rows; next: their choices.
int run_pass(LayeredModel* m, const dsk_step_entry* e, const std::vector<Part>& parts, const std::vector<int>& want, int mode, float* out, int32_t* next,
             const float* coins) {
  int rows = 0;
  bool single = true;
  for (const Part& p : parts) {
    rows += p.len;
    single &= p.len == 1;
  }
  const bool few = single && rows <= FEW;
  DescBuf& d = few ? m->small : m->big;
  SeqDesc* sd = reinterpret_cast<SeqDesc*>(d.host);
  int *tok = reinterpret_cast<int*>(d.host + d.o_tok), *row = reinterpret_cast<int*>(d.host + d.o_row), *wn = reinterpret_cast<int*>(d.host + d.o_want),
      *tile = reinterpret_cast<int*>(d.host + d.o_tile), *chunk = reinterpret_cast<int*>(d.host + d.o_chunk), *lone = reinterpret_cast<int*>(d.host + d.o_single);
  int r = 0, nt = 0, nc = 0, ns = 0, keys = 0, max_hist = 0;
  for (size_t i = 0; i < parts.size(); ++i) {
    const Part& p = parts[i];
    Seq& q = m->seqs[e[p.entry].seq];
    const int hist = older_keys(m, q.pos);
    sd[i] = {q.base, r, p.len, q.pos, q.flip, nc, keys, p.len > 1 ? hist : 0};
    if (p.len == 1) {
      lone[ns++] = (int)i;
    } else {
      keys += hist + p.len;
      max_hist = std::max(max_hist, hist);
    }
    for (int t = 0; t < p.len; ++t) {
      tok[r + t] = e[p.entry].tokens[p.first + t];
      row[r + t] = (int)i;
    }
    for (int t = 0; t < p.len; t += 64, ++nt) {
      tile[2 * nt] = (int)i;
      tile[2 * nt + 1] = t;
    }
    for (int t = 0; t < p.len; t += RECUR_CHUNK, ++nc) {
      chunk[2 * nc] = (int)i;
      chunk[2 * nc + 1] = t;
    }
    r += p.len;
  }
  for (size_t i = 0; i < want.size(); ++i) wn[i] = want[i];
  hipStream_t st = m->ctx->stream;
  const int nw = (int)want.size();
  PassDesc p = pass_desc(d, rows, (int)parts.size(), nw, nt, nc);
  p.n_single = ns;
  p.key_rows = keys;
  p.max_hist = max_hist;
  m->last_rows = rows;
  if (few) {
    if (mode == OUT_SAMPLE) {  // (sp_host's temperature and top_p were set by the caller)
      for (int i = 0; i < nw; ++i) m->sp_host[i].coin = coins[i];
    }
    int need = 1;  // parts of the longest chunk of keys any sequence has now; graphs differ by it
    for (const LayerSpec& l : m->s.layers)
      for (const Part& q : parts)
        if (l.has_attn) need = std::max(need, m->seqs[e[q.entry].seq].pos % l.attn.chunk / ATTN_SPLIT_KEYS + 1);
        else if (l.has_latent) need = std::max(need, std::min(m->seqs[e[q.entry].seq].pos, l.latent.window - 1) / latent_keys(m->f32) + 1);
    int lg = 0;
    while ((1 << lg) < need) ++lg;
    m->splits = 1 << lg;
    Graph& g = m->graphs[((lg * 32 + rows) * 32 + nw) * 4 + (nw ? mode : OUT_NONE)];
    if (!m->use_graph || m->trace || !g.primed) {  // the first pass of a kind runs eagerly, the second is captured
      g.primed = true;
      DSK_TRY(run_few(m, p, mode));
    } else {
      if (!g.exec) {
        hipGraph_t gr = nullptr;
        HIP_TRY(hipStreamBeginCapture(st, hipStreamCaptureModeThreadLocal));
        const int rc = run_few(m, p, mode);
        const hipError_t ec = hipStreamEndCapture(st, &gr);
        hipError_t ei = hipSuccess;
        if (rc == DSK_OK && ec == hipSuccess) ei = hipGraphInstantiate(&g.exec, gr, nullptr, nullptr, 0);
        if (gr) hipGraphDestroy(gr);
        if (rc != DSK_OK) return rc;
        if (ec != hipSuccess || ei != hipSuccess) {
          g.exec = nullptr;
          DSK_FAIL(DSK_ERR_HIP, "graph capture: %s", hipGetErrorString(ec != hipSuccess ? ec : ei));
        }
      }
      HIP_TRY(hipGraphLaunch(g.exec, st));
      m->graph_steps++;
    }
    HIP_TRY(hipStreamSynchronize(st));
    if (nw && mode == OUT_LOGITS) {
      if (out != m->logits_host) memcpy(out, m->logits_host, (size_t)nw * m->s.vocab * 4);
    } else if (nw) {
      memcpy(next, m->next_host, (size_t)nw * 4);
    }
  } else {
    m->splits = 1 << 30;  // (a mixer takes as many as its largest window has)
    DSK_TRY(run_body(m, d, p, false));
    const int block = mode == OUT_LOGITS ? LOGIT_ROWS : FEW;
    for (int i = 0; i < nw; i += block) {
      const int n = std::min(block, nw - i);
      DSK_TRY(run_head(m, i, n));
      if (mode == OUT_LOGITS) {
        HIP_TRY(hipMemcpy2DAsync(m->logits_host, (size_t)m->s.vocab * 4, m->logits, (size_t)m->ld_logits * 4, (size_t)m->s.vocab * 4, n, hipMemcpyDeviceToHost, st));
        HIP_TRY(hipStreamSynchronize(st));
        if (out + (size_t)i * m->s.vocab != m->logits_host) memcpy(out + (size_t)i * m->s.vocab, m->logits_host, (size_t)n * m->s.vocab * 4);
      } else {
        if (mode == OUT_SAMPLE)
          for (int k = 0; k < n; ++k) m->sp_host[k].coin = coins[i + k];
        DSK_TRY(run_choice(m, n, mode));
        HIP_TRY(hipStreamSynchronize(st));
        memcpy(next + i, m->next_host, (size_t)n * 4);
      }
    }
    HIP_TRY(hipStreamSynchronize(st));  // (the descriptor buffer is free again)
  }
  HIP_TRY(hipGetLastError());
  for (const Part& q : parts) {
    Seq& s = m->seqs[e[q.entry].seq];
    s.pos += q.len;
    s.flip ^= 1;
  }
  return DSK_OK;
}

int check_seq(LayeredModel* m, int32_t s) {
  if (s < 0 || s >= (int)m->seqs.size() || !m->seqs[s].live) DSK_FAIL(DSK_ERR_INVALID, "sequence %d is not open", s);
  return DSK_OK;
}

// A step in passes of at most `piece` rows.  Only an entry's last part may want its last row (modes ARGMAX / SAMPLE).
int run_step(LayeredModel* m, const dsk_step_entry* e, int n, int mode, float* out, int32_t* next, const float* coins) {
  HIP_TRY(hipSetDevice(m->ctx->device));
  for (int i = 0; i < n; ++i) DSK_TRY(check_seq(m, e[i].seq));
  std::vector<Part> parts;
  std::vector<int> want, want_entry;
  int rows = 0, keys = 0;  // keys: rows of the key workspace (latent attention)
  auto flush = [&]() -> int {
    if (parts.empty()) return DSK_OK;
    std::vector<int32_t> nx(want.size());
    std::vector<float> cn;
    if (coins)
      for (int w : want_entry) cn.push_back(coins[w]);
    DSK_TRY(run_pass(m, e, parts, want, mode, out, nx.data(), cn.data()));
    if (mode == OUT_LOGITS) out += want.size() * (size_t)m->s.vocab;
    else
      for (size_t i = 0; i < want.size(); ++i) next[want_entry[i]] = nx[i];
    parts.clear();
    want.clear();
    want_entry.clear();
    rows = keys = 0;
    return DSK_OK;
  };
  for (int i = 0; i < n; ++i) {
    for (int t = 1; mode == OUT_LOGITS && t < e[i].n_want; ++t)
      if (e[i].want[t] <= e[i].want[t - 1]) DSK_FAIL(DSK_ERR_UNSUPPORTED, "step: the wanted places must ascend");
    for (int done = 0; done < e[i].n_tokens;) {
      const int len = std::min(e[i].n_tokens - done, m->piece - rows);
      const int k = m->max_window && len > 1 ? older_keys(m, m->seqs[e[i].seq].pos) + len : 0;
      if (len == 0 || (rows && keys + k > m->key_cap && k)) {  // (behind a flush everything fits)
        DSK_TRY(flush());
        continue;
      }
      keys += k;
      parts.push_back({i, done, len});
      if (mode == OUT_LOGITS) {
        for (int w = 0; w < e[i].n_want; ++w)
          if (e[i].want[w] >= done && e[i].want[w] < done + len) want.push_back(rows + e[i].want[w] - done);
      } else if (done + len == e[i].n_tokens) {
        want.push_back(rows + len - 1);
        want_entry.push_back(i);
      }
      rows += len;
      done += len;
    }
  }
  return flush();
}

// ---- the family table --------------------------------------------------------------------------------------
int l_destroy(dsk_model* h) {
  LayeredModel* m = lm(h);
  hipSetDevice(m->ctx->device);
  hipStreamSynchronize(m->ctx->stream);
  for (auto& g : m->graphs)
    if (g.second.exec) hipGraphExecDestroy(g.second.exec);
  for (void* p : m->dev) hipFree(p);
  for (void* p : m->slabs) hipFree(p);
  for (void* p : {(void*)m->sp_host, (void*)m->logits_host, (void*)m->next_host, (void*)m->big.host, (void*)m->small.host})
    if (p) hipHostFree(p);
  dsk_ctx* ctx = m->ctx;
  delete m;
  ctx_model_released(ctx);
  return DSK_OK;
}
int l_vocab(const dsk_model* h) { return lm(h)->s.vocab; }

int l_seq_open(dsk_model* h, int32_t* seq) {
  LayeredModel* m = lm(h);
  HIP_TRY(hipSetDevice(m->ctx->device));
  for (int pass = 0; pass < 2; ++pass) {
    for (size_t i = 0; i < m->seqs.size(); ++i)
      if (!m->seqs[i].live) {
        m->seqs[i].live = true;
        m->seqs[i].pos = m->seqs[i].flip = 0;  // position 0: kernels start from zero state and read nothing of the arena
        *seq = (int32_t)i;
        return DSK_OK;
      }
    if (pass == 0) {  // another slab of arenas: up to 8, at most about 256 MiB
      const size_t n = std::max<size_t>(1, std::min<size_t>(8, ((size_t)256 << 20) / m->seq_bytes));
      void* p = nullptr;
      HIP_TRY(hipMalloc(&p, n * m->seq_bytes));
      m->slabs.push_back(p);
      m->cache_bytes += (double)(n * m->seq_bytes);
      for (size_t i = 0; i < n; ++i) {
        Seq s;
        s.base = (char*)p + i * m->seq_bytes;
        m->seqs.push_back(s);
      }
    }
  }
  DSK_FAIL(DSK_ERR_NOMEM, "seq_open: no room for another sequence");
}
int l_seq_close(dsk_model* h, int32_t s) {
  LayeredModel* m = lm(h);
  DSK_TRY(check_seq(m, s));
  m->seqs[s].live = false;
  return DSK_OK;
}
int l_seq_pos(dsk_model* h, int32_t s, int32_t* pos) {
  LayeredModel* m = lm(h);
  DSK_TRY(check_seq(m, s));
  *pos = m->seqs[s].pos;
  return DSK_OK;
}
int l_step(dsk_model* h, const dsk_step_entry* e, int n, float* logits) { return run_step(lm(h), e, n, OUT_LOGITS, logits, nullptr, nullptr); }
int l_step_sample(dsk_model* h, const dsk_step_entry* e, int n, float temperature, float top_p, const float* coins, int32_t* next) {
  LayeredModel* m = lm(h);
  for (int i = 0; i < FEW; ++i) {
    m->sp_host[i].temperature = temperature;
    m->sp_host[i].top_p = top_p;
    m->sp_host[i].prob_index = -1;
  }
  return run_step(m, e, n, temperature == 0.0f ? OUT_ARGMAX : OUT_SAMPLE, nullptr, next, temperature == 0.0f ? nullptr : coins);
}

// the single-sequence calls run on a sequence of the model's own; position 0 starts it anew
int own_seq(LayeredModel* m, const int32_t* tokens, int n, int pos) {
  for (int i = 0; i < n; ++i)
    if (tokens[i] < 0 || tokens[i] >= m->s.vocab) DSK_FAIL(DSK_ERR_INVALID, "forward: token %d out of range", tokens[i]);
  dsk_model* h = reinterpret_cast<dsk_model*>(m);
  if (m->own_seq < 0) DSK_TRY(l_seq_open(h, &m->own_seq));
  Seq& s = m->seqs[m->own_seq];
  if (pos == 0) s.pos = s.flip = 0;
  if (pos != s.pos) DSK_FAIL(DSK_ERR_STATE, "forward: position %d, but the sequence stands at %d (a recurrent state cannot go back)", pos, s.pos);
  return DSK_OK;
}
int l_hydrate(dsk_model* h, const int32_t* tokens, int n, int pos0, int mode, float* host_logits) {
  LayeredModel* m = lm(h);
  if (!tokens || n < 1 || pos0 < 0) DSK_FAIL(DSK_ERR_INVALID, "hydrate: %d tokens at pos %d", n, pos0);
  if (mode != DSK_MODE_HYDRATE_KV_CACHE && mode != DSK_MODE_OUTPUT_LOGITS) DSK_FAIL(DSK_ERR_INVALID, "hydrate: bad mode %d", mode);
  if (mode == DSK_MODE_OUTPUT_LOGITS && !host_logits) DSK_FAIL(DSK_ERR_INVALID, "hydrate: OUTPUT_LOGITS needs a logits buffer");
  DSK_TRY(own_seq(m, tokens, n, pos0));
  const int32_t last = n - 1;
  const dsk_step_entry e = {m->own_seq, n, tokens, mode == DSK_MODE_OUTPUT_LOGITS ? 1 : 0, &last};
  return run_step(m, &e, 1, OUT_LOGITS, host_logits, nullptr, nullptr);
}
int l_forward(dsk_model* h, int token, int pos, int mode, float* host_logits) {
  const int32_t t = token;
  return l_hydrate(h, &t, 1, pos, mode, host_logits);
}
int l_choose(LayeredModel* m, int token, int pos, int mode, float temperature, float top_p, float coin, int prob_index, int32_t* next) {
  const int32_t t = token;
  DSK_TRY(own_seq(m, &t, 1, pos));
  for (int i = 0; i < FEW; ++i) {
    m->sp_host[i].temperature = temperature;
    m->sp_host[i].top_p = top_p;
    m->sp_host[i].prob_index = prob_index;
  }
  const dsk_step_entry e = {m->own_seq, 1, &t, 0, nullptr};
  return run_step(m, &e, 1, mode, nullptr, next, &coin);
}
int l_forward_argmax(dsk_model* h, int token, int pos, int32_t* next) {
  if (!next) DSK_FAIL(DSK_ERR_INVALID, "forward_argmax: null output");
  return l_choose(lm(h), token, pos, OUT_ARGMAX, 0.f, 0.f, 0.f, -1, next);
}
int l_forward_sample(dsk_model* h, int token, int pos, float temperature, float top_p, float coin, int32_t* next) {
  if (!next) DSK_FAIL(DSK_ERR_INVALID, "forward_sample: null output");
  return l_choose(lm(h), token, pos, temperature == 0.0f ? OUT_ARGMAX : OUT_SAMPLE, temperature, top_p, coin, -1, next);
}
int l_forward_prob(dsk_model* h, int token, int pos, int index, float* prob) {
  if (!prob || index < 0 || index >= lm(h)->s.vocab) DSK_FAIL(DSK_ERR_INVALID, "forward_prob: bad index %d", index);
  int32_t bits = 0;
  DSK_TRY(l_choose(lm(h), token, pos, OUT_SAMPLE, 1.f, 1.f, 0.f, index, &bits));
  memcpy(prob, &bits, 4);
  return DSK_OK;
}
float* l_host_logits(dsk_model* h) { return lm(h)->logits_host; }
int l_set_graph(dsk_model* h, int on) {
  lm(h)->use_graph = on != 0;
  return DSK_OK;
}
int l_set_trace(dsk_model* h, int on) {
  LayeredModel* m = lm(h);
  HIP_TRY(hipSetDevice(m->ctx->device));
  if (on && !m->trace_x) DSK_TRY(dev_alloc_n(m, &m->trace_x, m->L.size() * (size_t)m->piece * m->s.width));
  m->trace = on != 0;
  return DSK_OK;
}
int l_trace_row(dsk_model* h, int layer, int row, float* x) {
  LayeredModel* m = lm(h);
  if (!m->trace || !x) DSK_FAIL(DSK_ERR_STATE, "trace: dsk_model_set_trace(1) before the step");
  if (layer < 0 || layer >= (int)m->L.size() || row < 0 || row >= m->last_rows) DSK_FAIL(DSK_ERR_INVALID, "trace: layer %d row %d (the last pass held %d)", layer, row, m->last_rows);
  HIP_TRY(hipSetDevice(m->ctx->device));
  HIP_TRY(hipMemcpy(x, m->trace_x + ((size_t)layer * m->piece + row) * m->s.width, (size_t)m->s.width * 4, hipMemcpyDeviceToHost));
  return DSK_OK;
}
int l_get_trace_x(dsk_model* h, int layer, float* x) { return l_trace_row(h, layer, lm(h)->last_rows - 1, x); }
int l_get_info(dsk_model* h, const char* key, int* value) {
  LayeredModel* m = lm(h);
  if (!key || !value) DSK_FAIL(DSK_ERR_INVALID, "get_info: null argument");
  const std::string k(key);
  if (k == "graph_captured") {
    *value = 0;
    for (auto& g : m->graphs) *value += g.second.exec != nullptr;
  } else if (k == "graph_steps") *value = m->graph_steps;
  else if (k == "fused_decode_layers") *value = (int)std::min<long long>(m->fused_layers, 0x7fffffff);
  else if (k == "layers") *value = (int)m->L.size();
  else if (k == "width") *value = m->s.width;
  else if (k == "piece_tokens") *value = m->piece;
  else if (k == "sequence_kb") *value = (int)(m->seq_bytes >> 10);
  else if (k == "live_sequences") {
    *value = 0;
    for (auto& s : m->seqs) *value += s.live;
  } else if (k == "sequence_slots") *value = (int)m->seqs.size();
  else DSK_FAIL(DSK_ERR_INVALID, "get_info: unknown key '%s'", key);
  return DSK_OK;
}
// bytes one decoded token of one sequence reads (and, of the recurrent state, writes)
double l_active_bytes(const dsk_model* h, int pos) {
  const LayeredModel* m = lm(h);
  double b = 2.0 * m->s.width + 2.0 * (double)m->head.elems();
  for (size_t i = 0; i < m->L.size(); ++i) {
    const LayerSpec& l = m->s.layers[i];
    const LayerW& w = m->L[i];
    b += 2.0 * (double)w.proj.elems();
    if (l.has_attn)
      b += 2.0 * (double)w.a_o.elems() + (double)(pos % l.attn.chunk) * l.attn.kv_heads * (l.attn.dim + l.attn.vdim) * m->elem();
    if (l.has_mlstm) b += 2.0 * (double)w.m_o.elems() + 8.0 * l.mlstm.heads * l.mlstm.dim * (l.mlstm.vdim + 1);
    if (l.has_delta) b += 2.0 * (double)(w.d_o.elems() + w.d_low2.elems()) + 8.0 * l.delta.heads * l.delta.dim * l.delta.vdim;
    if (l.has_wkv) b += 2.0 * (double)(w.w_o.elems() + w.w_low2.elems()) + 8.0 * l.wkv.heads * l.wkv.dim * l.wkv.dim;
    if (l.has_latent)
      b += 2.0 * (double)(w.l_uq.elems() + w.l_abs.elems() + (size_t)l.latent.heads * w.vdim_p * w.rank_p + w.l_o.elems()) +
           (double)std::min(pos + 1, l.latent.window) * (w.rank_p + w.rot_p) * m->elem();
    if (l.has_dense) b += 2.0 * (double)(w.ff_up.elems() + w.ff_down.elems());
    if (l.has_moe) {
      b += 2.0 * l.moe.top * (double)(w.e_up.stride + w.e_down.stride);
      if (l.moe.shared_ff) b += 1024.0 * ((double)w.e_up.shared_kt * w.e_up.shared_rt + (double)w.e_down.shared_kt * w.e_down.shared_rt);
    }
  }
  return b;
}
double l_device_bytes(const dsk_model* h) { return lm(h)->weight_bytes + lm(h)->scratch_bytes + lm(h)->cache_bytes; }

const Family layered_family = {"layered",     l_destroy,    l_vocab,       l_forward,      l_hydrate,      l_forward_argmax, l_forward_sample, l_forward_prob, l_host_logits, l_set_graph, l_set_trace,
                               l_get_trace_x, l_trace_row,  l_get_info,    l_active_bytes, l_device_bytes, l_seq_open,       l_seq_close,      l_seq_pos,      l_step,        l_step_sample};

// ---- opening -------------------------------------------------------------------------------------------------
int set_options(LayeredModel* m, const char* options) {
  for (const char* p = options; p && *p;) {
    const char* e = strchr(p, ',');
    const std::string kv(p, e ? (size_t)(e - p) : strlen(p));
    const size_t eq = kv.find('=');
    if (eq == std::string::npos || eq == 0 || eq + 1 >= kv.size()) DSK_FAIL(DSK_ERR_INVALID, "open: malformed option '%s' (key=value expected)", kv.c_str());
    const std::string k = kv.substr(0, eq);
    const int v = atoi(kv.c_str() + eq + 1);
    if (k == "piece_tokens") {
      if (v < FEW || v > 16384) DSK_FAIL(DSK_ERR_INVALID, "open: piece_tokens %d (16 .. 16384)", v);
      m->piece = v;
    } else if (k == "decode_graph") m->use_graph = v != 0;
    else if (k == "fused_decode") m->fused_decode = v != 0;
    else if (k == "chunk_scan") m->chunk_scan = v != 0;
    else if (k == "prompt_tile") {
      if (v != 0 && v != 128 && v != 256) DSK_FAIL(DSK_ERR_INVALID, "open: prompt_tile %d (0, 128, 256)", v);
      m->tile = v;
    }
    else DSK_FAIL(DSK_ERR_INVALID, "open: unknown option '%s'", k.c_str());
    p = e ? e + 1 : nullptr;
  }
  return DSK_OK;
}
int load_all(LayeredModel* m, Checkpoint* ck, uint64_t seed) {
  const LayeredSpec& s = m->s;
  Weights W{m, ck, seed};
  uint16_t* p;
  DSK_TRY(dev_alloc_n(m, &m->embed, (size_t)s.vocab * s.width, true));
  DSK_TRY(W.get(s.embed, s.vocab, s.width, &p));
  HIP_TRY(hipMemcpyAsync(m->embed, p, (size_t)s.vocab * s.width * 2, hipMemcpyDeviceToDevice, m->ctx->stream));
  DSK_TRY(W.floats(s.final_norm, 0, s.width, &m->final_norm));
  DSK_TRY(W.matrix(s.head, s.vocab, s.width, &m->head));
  m->L.resize(s.layers.size());
  for (size_t i = 0; i < m->L.size(); ++i) DSK_TRY(load_layer(W, m, s.layers[i], m->L[i]));
  layout_state(m);
  DSK_TRY(alloc_work(m));
  HIP_TRY(hipStreamSynchronize(m->ctx->stream));
  HIP_TRY(hipGetLastError());
  return DSK_OK;
}
int open_model(dsk_ctx* ctx, const JVal& config, Checkpoint* ck, int dtype, const char* options, uint64_t seed, dsk_model** out) {
  LayeredSpec spec;
  DSK_TRY(layered_parse(config, &spec));
  if (ctx->closing) DSK_FAIL(DSK_ERR_STATE, "model_open: the context has been destroyed");
  HIP_TRY(hipSetDevice(ctx->device));
  LayeredModel* m = new LayeredModel();
  m->family = &layered_family;
  m->ctx = ctx;
  m->s = spec;
  m->f32 = dtype == DSK_DTYPE_F32;
  ctx->live_models++;
  int r = set_options(m, options);
  if (r == DSK_OK) r = load_all(m, ck, seed);
  if (r != DSK_OK) {
    const std::string keep = dsk_last_error();
    l_destroy(reinterpret_cast<dsk_model*>(m));
    dsk_restore_error(keep.c_str());
    return r;
  }
  *out = reinterpret_cast<dsk_model*>(m);
  return DSK_OK;
}
int open_dir(dsk_ctx* ctx, const char* dir, int dtype, const char* options, dsk_model** out) {
  std::string text;
  JVal config;
  DSK_TRY(read_text_file(std::string(dir) + "/config.json", &text));
  if (!json_parse(text, &config)) DSK_FAIL(DSK_ERR_INVALID, "loader: config.json is not JSON");
  Checkpoint ck;
  DSK_TRY(open_checkpoint_file((std::string(dir) + "/model.safetensors").c_str(), ck));
  return open_model(ctx, config, &ck, dtype, options, 0, out);
}
FamilyLoader layered_loader(layered_design_known, open_dir);

}  // namespace

extern "C" int dsk_config_check(const char* config_json) {
  if (!config_json) DSK_FAIL(DSK_ERR_INVALID, "config_check: null argument");
  JVal config;
  if (!json_parse(config_json, &config)) DSK_FAIL(DSK_ERR_INVALID, "config_check: the configuration is not JSON");
  LayeredSpec spec;
  return layered_parse(config, &spec);
}

extern "C" int dsk_model_open_synthetic(dsk_ctx* ctx, const char* config_json, int dtype, const char* options, uint64_t seed, dsk_model** out) {
  if (!ctx || !config_json || !out) DSK_FAIL(DSK_ERR_INVALID, "model_open_synthetic: null argument");
  if (dtype != DSK_DTYPE_BF16 && dtype != DSK_DTYPE_F32) DSK_FAIL(DSK_ERR_INVALID, "model_open_synthetic: dtype %d", dtype);
  *out = nullptr;
  JVal config;
  if (!json_parse(config_json, &config)) DSK_FAIL(DSK_ERR_INVALID, "model_open_synthetic: the configuration is not JSON");
  return open_model(ctx, config, nullptr, dtype, options, seed + 1, out);
}
