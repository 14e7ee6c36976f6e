// layered.h -- layered models: designs whose configuration lists their layers, each made of mechanisms (kinds of attention,
// recurrent mixers, a router with experts) with their constants as parameters.  layered_config.cpp turns a configuration into a
// LayeredSpec; layered_model.cpp loads the weights a spec names, keeps the sequences' state and runs steps.
#pragma once
#include "checkpoint.h"
#include "context.h"
#include "layered_kernels.h"

#include <map>
#include <string>
#include <vector>

// ---- what a design is made of ----
struct RotSpec {       // rotary positions on the first `dims` dimensions; optional YaRN frequencies.  How dimensions pair up (2i with
  int dims = 0;        // 2i + 1, or i with i + dims / 2) belongs to the mechanism
  double base = 10000.0;
  bool scaled = false;
  double factor = 1.0, original = 0.0, fast = 32.0, slow = 1.0;
};
struct AttnSpec {      // softmax attention inside chunks, q and k RMS-normed per head after rotation
  int heads = 0, kv_heads = 0, dim = 0, vdim = 0, chunk = 0;
  double scale = 1.0;
  RotSpec rot;
  std::string name;    // tensors "<name>.q" ...
};
struct MlstmSpec {
  int heads = 0, dim = 0, vdim = 0;
  double gate_cap = 0.0, floor_eps = 1e-6;
  std::string name;
};
struct DeltaSpec {     // gated delta rule
  int heads = 0, kv_heads = 0, dim = 0, vdim = 0, taps = 0;
  double unit_eps = 1e-6;
  bool head_decay = false;  // one decay per head from ".a"; else one per key channel from the low-rank pair ".a1", ".a2"
  bool silu_gate = false;   // silu of ".g" behind it; else the sigmoid of the low-rank pair ".g1", ".g2"
  std::string name;
};
struct WkvSpec {       // time mixing: every projection reads its own blend of the token's input with the previous one's; decays per key
  int heads = 0, dim = 0;  // channel, a bonus for the current token
  std::string name;
};
struct LatentSpec {    // softmax attention in a sliding window; keys and values come from one normed latent and one rotated part per token
  int heads = 0, dim = 0, rot_dim = 0, vdim = 0, q_rank = 0, kv_rank = 0, window = 0;
  double scale = 1.0;
  RotSpec rot;         // of the rot_dim part, dimension i with i + dims / 2
  std::string name;
};
struct DenseSpec {     // down(xielu(up(h)))
  int ff = 0;
  std::string name;
};
struct MoeSpec {
  int experts = 0, top = 0, ff = 0, shared_ff = 0;  // shared_ff = 0: no shared expert
  double limit = 0.0, shared_limit = 0.0;
  double alpha = 1.702, up_offset = 1.0;            // min(g, limit) * sigmoid(alpha g) * (clamp(u) + up_offset)
  std::string name;
};
// Two forms of a layer.  Parallel: x += mixers(norm(x)) + ff(norm(x)).  Sandwich: x += post(mixer(in(norm(x)))), then the same around the
// feed-forward with norms and convolutions of its own; in(h) = h + a causal convolution of h over time, `taps` taps per channel.
struct LayerSpec {
  std::string norm;
  bool has_attn = false, has_mlstm = false, has_delta = false, has_wkv = false, has_latent = false, has_moe = false, has_dense = false;
  AttnSpec attn;
  MlstmSpec mlstm;
  DeltaSpec delta;
  WkvSpec wkv;
  LatentSpec latent;
  MoeSpec moe;
  DenseSpec dense;
  std::string pair_a, pair_b;  // two mixers: half the sum of their outputs, each RMS-normed with this weight (attention, recurrence)
  bool sandwich = false;
  std::string post, conv, ff_norm, ff_post, ff_conv;  // (sandwich)
  int taps = 1;
};
struct LayeredSpec {
  std::string design, embed, final_norm, head;
  int width = 0, vocab = 0;
  double eps = 1e-6, norm_offset = 0.0, softcap = 0.0, logit_scale = 1.0;  // softcap = 0: none
  std::vector<LayerSpec> layers;
};
bool layered_design_known(const char* architecture);
int layered_parse(const JVal& config, LayeredSpec* out);
// frequencies of the pairs and the factor on cos and sin
void rot_frequencies(const RotSpec& r, std::vector<float>* freq, float* amp);
