// layered_config.cpp -- configurations of layered designs (layered.h): one parser per design, found by its name.
#include "layered.h"

#include <math.h>
#include <string.h>

#include <algorithm>

namespace {

// typed access to a JSON object; the first missing or ill-typed key is what the error says
struct Obj {
  const JVal* v;
  std::string path;
  std::string* bad;
  Obj(const JVal* v_, const std::string& p, std::string* b) : v(v_), path(p), bad(b) {
    if (!v || v->kind != JVal::OBJ) fail("is not an object");
  }
  void fail(const std::string& why) const {
    if (bad->empty()) *bad = path + " " + why;
  }
  bool has(const char* k) const {
    const JVal* x = v && v->kind == JVal::OBJ ? v->get(k) : nullptr;
    return x && x->kind != JVal::NUL;
  }
  Obj at(const char* k) const { return Obj(has(k) ? v->get(k) : nullptr, path + "." + k, bad); }
  double num(const char* k) const {
    const JVal* x = has(k) ? v->get(k) : nullptr;
    if (!x || x->kind != JVal::NUM || !std::isfinite(x->num)) {
      fail(std::string("has no number '") + k + "'");
      return 0.0;
    }
    return x->num;
  }
  int size(const char* k) const {  // a positive integer
    const double d = num(k);
    if (bad->empty() && (d < 1 || d > 1e9 || d != (double)(int)d)) fail(std::string("'") + k + "' is not a positive integer");
    return bad->empty() ? (int)d : 1;
  }
  std::string str(const char* k) const {
    const JVal* x = has(k) ? v->get(k) : nullptr;
    if (!x || x->kind != JVal::STR) {
      fail(std::string("has no string '") + k + "'");
      return "";
    }
    return x->str;
  }
};

RotSpec parse_rot(const Obj& o) {
  RotSpec r;
  r.dims = o.size("dims");
  r.base = o.num("base");
  if (r.dims & 1) o.fail("'dims' is odd");
  if (o.has("scaling")) {
    const Obj s = o.at("scaling");
    r.scaled = true;
    r.factor = s.num("factor");
    r.original = s.num("original");
    r.fast = s.num("fast");
    r.slow = s.num("slow");
    if (s.bad->empty() && (r.factor <= 0 || r.original <= 0 || r.fast <= 0 || r.slow <= 0)) s.fail("has a factor that is not positive");
  }
  return r;
}
void check_groups(const Obj& o, int heads, int kv_heads) {
  if (o.bad->empty() && heads % kv_heads) o.fail("'heads' is not a multiple of 'kv_heads'");
}
AttnSpec parse_attn(const Obj& o, const std::string& name) {
  AttnSpec a;
  a.name = name;
  a.heads = o.size("heads");
  a.kv_heads = o.size("kv_heads");
  a.dim = o.size("dim");
  a.vdim = o.size("vdim");
  a.chunk = o.at("mask").size("size");
  a.scale = o.num("scale");
  if (o.has("rot")) a.rot = parse_rot(o.at("rot"));
  if (a.rot.dims > a.dim) o.fail("rotates more dimensions than a head has");
  check_groups(o, a.heads, a.kv_heads);
  return a;
}
MlstmSpec parse_mlstm(const Obj& o, const std::string& name) {
  MlstmSpec a;
  a.name = name;
  a.heads = o.size("heads");
  a.dim = o.size("dim");
  a.vdim = o.size("vdim");
  a.gate_cap = o.num("gate_cap");
  if (o.bad->empty() && a.gate_cap <= 0) o.fail("'gate_cap' is not positive");
  return a;
}
DeltaSpec parse_delta(const Obj& o, const std::string& name) {
  DeltaSpec a;
  a.name = name;
  a.heads = o.size("heads");
  a.kv_heads = o.size("kv_heads");
  a.dim = o.size("dim");
  a.vdim = o.size("vdim");
  a.taps = o.size("conv");
  check_groups(o, a.heads, a.kv_heads);
  return a;
}
WkvSpec parse_wkv(const Obj& o, const std::string& name) {
  WkvSpec a;
  a.name = name;
  a.heads = o.size("heads");
  a.dim = o.size("dim");
  return a;
}
LatentSpec parse_latent(const Obj& o, const std::string& name) {
  LatentSpec a;
  a.name = name;
  a.heads = o.size("heads");
  a.dim = o.size("dim");
  a.rot_dim = o.size("rot_dim");
  a.vdim = o.size("vdim");
  a.q_rank = o.size("q_rank");
  a.kv_rank = o.size("kv_rank");
  a.window = o.at("mask").size("size");
  a.scale = o.num("scale");
  a.rot = parse_rot(o.at("rot"));
  if (o.bad->empty() && a.rot.dims > a.rot_dim) o.fail("rotates more dimensions than 'rot_dim'");
  return a;
}
DenseSpec parse_dense(const Obj& o, const std::string& name) {
  DenseSpec d;
  d.name = name;
  if (o.str("kind") != "dense") o.fail("'kind' is not known");
  d.ff = o.size("ff");
  return d;
}
MoeSpec parse_moe(const Obj& o, const std::string& name) {
  MoeSpec m;
  m.name = name;
  if (o.str("kind") != "moe") o.fail("'kind' is not known");
  m.experts = o.at("router").size("experts");
  m.top = o.at("router").size("top");
  m.ff = o.at("expert").size("ff");
  m.limit = o.at("expert").num("limit");
  if (o.has("shared")) {
    m.shared_ff = o.at("shared").size("ff");
    m.shared_limit = o.at("shared").num("limit");
  }
  if (o.bad->empty() && m.top > m.experts) o.fail("'top' is larger than 'experts'");
  return m;
}

// Timerax: parallel residual with one norm (weight around zero) per layer; layers of two kinds - "parallel" (chunked attention
// beside an mLSTM, half the sum of their normed outputs) and "channel_delta" (gated delta rule, a decay per key channel) - and
// mixtures of clamped-GLU experts.
void parse_timerax(const Obj& root, LayeredSpec* s) {
  s->width = root.size("width");
  s->vocab = root.size("vocab");
  s->eps = root.at("norm").num("eps");
  s->norm_offset = 1.0;
  if (root.has("logit_softcap")) {
    s->softcap = root.num("logit_softcap");
    if (s->softcap <= 0) root.fail("'logit_softcap' is not positive");
  }
  s->embed = "embed";
  s->final_norm = "final.norm";
  s->head = "head";
  const JVal* layers = root.v->get("layers");
  if (!layers || layers->kind != JVal::ARR || layers->arr.empty()) {
    root.fail("lists no layers");
    return;
  }
  for (size_t i = 0; i < layers->arr.size(); ++i) {
    const Obj o(&layers->arr[i], root.path + ".layers[" + std::to_string(i) + "]", root.bad);
    LayerSpec l;
    const std::string pre = "l" + std::to_string(i) + ".", type = o.str("type");
    l.norm = pre + "norm1";
    const Obj mix = o.at("mixer");
    if (type == "parallel") {
      l.has_attn = l.has_mlstm = true;
      l.attn = parse_attn(mix.at("left"), pre + "mix.left");
      l.mlstm = parse_mlstm(mix.at("right"), pre + "mix.right");
      l.pair_a = pre + "mix.left.out";
      l.pair_b = pre + "mix.right.out";
    } else if (type == "channel_delta") {
      l.has_delta = true;
      l.delta = parse_delta(mix, pre + "mix");
    } else {
      o.fail("has the unknown type '" + type + "'");
    }
    if (o.has("mlp")) {
      l.has_moe = true;
      l.moe = parse_moe(o.at("mlp"), pre + "mlp");
    }
    s->layers.push_back(l);
  }
}

// Ranutar: sandwich layers (a norm with its weight around zero before and behind each sublayer, a causal convolution in front of it)
// of three kinds - "wkv" (time mixing), "delta" (gated delta rule, a decay per head), "latent_attention" (sliding window) - and dense
// feed-forwards.
void parse_ranutar(const Obj& root, LayeredSpec* s) {
  s->width = root.size("width");
  s->vocab = root.size("vocab");
  s->eps = root.at("norm").num("eps");
  s->norm_offset = 1.0;
  s->logit_scale = root.num("logit_scale");
  s->embed = "embed";
  s->final_norm = "final.norm";
  s->head = "head";
  const int taps = root.at("canon").size("taps");
  const JVal* layers = root.v->get("layers");
  if (!layers || layers->kind != JVal::ARR || layers->arr.empty()) {
    root.fail("lists no layers");
    return;
  }
  for (size_t i = 0; i < layers->arr.size(); ++i) {
    const Obj o(&layers->arr[i], root.path + ".layers[" + std::to_string(i) + "]", root.bad);
    LayerSpec l;
    const std::string pre = "l" + std::to_string(i) + ".", type = o.str("type");
    l.sandwich = true;
    l.taps = taps;
    l.norm = pre + "norm1";
    l.post = pre + "norm1b";
    l.conv = pre + "canon1";
    const Obj mix = o.at("mixer");
    if (type == "wkv") {
      l.has_wkv = true;
      l.wkv = parse_wkv(mix, pre + "mix");
    } else if (type == "delta") {
      l.has_delta = true;
      l.delta = parse_delta(mix, pre + "mix");
      l.delta.head_decay = l.delta.silu_gate = true;
    } else if (type == "latent_attention") {
      l.has_latent = true;
      l.latent = parse_latent(mix, pre + "mix");
    } else {
      o.fail("has the unknown type '" + type + "'");
    }
    if (o.has("mlp")) {
      l.has_dense = true;
      l.dense = parse_dense(o.at("mlp"), pre + "mlp");
      l.ff_norm = pre + "norm2";
      l.ff_post = pre + "norm2b";
      l.ff_conv = pre + "canon2";
    }
    s->layers.push_back(l);
  }
}

struct Design {
  const char* name;
  void (*parse)(const Obj& root, LayeredSpec* out);
};
const Design DESIGNS[] = {{"Timerax", parse_timerax}, {"Ranutar", parse_ranutar}};

}  // namespace

bool layered_design_known(const char* architecture) {
  for (const Design& d : DESIGNS)
    if (!strcmp(d.name, architecture)) return true;
  return false;
}

int layered_parse(const JVal& config, LayeredSpec* out) {
  std::string bad;
  const Obj root(&config, "config", &bad);
  const std::string name = root.str("architecture");
  if (bad.empty() && !layered_design_known(name.c_str())) DSK_FAIL(DSK_ERR_UNSUPPORTED, "config: unknown architecture '%s'", name.c_str());
  *out = LayeredSpec();
  out->design = name;
  for (const Design& d : DESIGNS)
    if (name == d.name) d.parse(root, out);
  if (!bad.empty()) DSK_FAIL(DSK_ERR_INVALID, "%s", bad.c_str());
  return DSK_OK;
}

// YaRN: pairs that turn often keep their frequency, pairs that turn less than `slow` times over the original context are divided by
// `factor`, a linear ramp over the pair index in between
void rot_frequencies(const RotSpec& r, std::vector<float>* freq, float* amp) {
  freq->resize(r.dims / 2);
  *amp = 1.f;
  double lo = 0, hi = 0;
  if (r.scaled) {
    auto index_of = [&](double turns) { return r.dims * log(r.original / (2 * M_PI * turns)) / (2 * log(r.base)); };
    lo = std::max(floor(index_of(r.fast)), 0.0);
    hi = std::min(ceil(index_of(r.slow)), (double)(r.dims - 1));
    *amp = (float)(0.1 * log(r.factor) + 1.0);
  }
  for (int i = 0; i < r.dims / 2; ++i) {
    double f = pow(r.base, -2.0 * i / r.dims);
    if (r.scaled) {
      const double ramp = std::min(std::max((i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
      f = f / r.factor * ramp + f * (1.0 - ramp);
    }
    (*freq)[i] = (float)f;
  }
}
