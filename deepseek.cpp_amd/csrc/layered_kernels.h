// layered_kernels.h -- launchers of the kernels behind layered models (layered.h); host-side argument blocks.
//
// Rows: a pass runs `rows` tokens, packed without padding, several sequences behind each other.  Pointers named *_t hold
// activations in the run's type (bf16 or float, f32 != 0); leading dimensions are in elements.
#pragma once
#include "dsk_internal.h"

// ---- what a pass knows about its sequences (device memory, filled by the host per pass) ----
struct SeqDesc {
  char* state;   // the sequence's arena
  int row0, len; // its rows in this pass
  int pos0;      // position of row0
  int flip;      // which copy of double-buffered state this pass reads (it writes the other)
  int chunk0;    // first of its recurrence chunks in PassDesc::chunk
  int key0, hist;  // portions of several tokens: rows of the key workspace (latent attention), `hist` older keys in front of the portion's
};
struct PassDesc {  // device pointers into one buffer
  const int* tokens;      // [rows]
  const int* row_seq;     // [rows] index into seqs
  const SeqDesc* seqs;
  const int* want;        // [n_want] rows whose logits are wanted
  const int* qtile;       // [n_qtiles][2]: sequence index, first row of the tile inside the sequence
  const int* chunk;       // [n_chunks][2]: sequence index, first row inside the sequence (RECUR_CHUNK rows each)
  const int* single;      // [n_single] sequences that bring one token
  int rows, n_seqs, n_want, n_qtiles, n_chunks, n_single;
  int key_rows, max_hist; // rows of the key workspace, the largest SeqDesc::hist
};

// ---- packed matrices ----
struct PackedMat {
  uint16_t* w = nullptr;  // fragments, row tile major: [row tiles][kt][64][8]
  int rows = 0, k = 0;    // logical
  int rt = 0, kt = 0;     // row tiles (padded to 8), k tiles (padded to 2)
  size_t elems() const { return (size_t)rt * kt * 512; }
};
// src [rows, k] row-major bf16 into the fragments of dst, at dst row `row0` and column `col0`; interleave >= 0: row r goes to row
// tile 2 * (r / 16) + interleave instead (pairs of tiles: gate, up); transpose: element (r, c) goes to dst row row0 + c, column col0 + r
int launch_pack(hipStream_t st, const uint16_t* src, int rows, int k, uint16_t* dst, int kt, int row0, int col0, int interleave, bool transpose = false);
int launch_widen(hipStream_t st, const uint16_t* src, float* dst, size_t n);  // bf16 -> f32
int launch_exp(hipStream_t st, float* x, int n);                             // in place
int launch_fill_random(hipStream_t st, uint16_t* dst, size_t n, float scale, uint64_t seed);  // bf16, uniform in +-scale
int launch_fill_random_f32(hipStream_t st, float* dst, size_t n, float scale, uint64_t seed);

// ---- matrix products: out[row, feature] = sum_k A[row, k] W[feature, k] ----
enum { LIN_STORE = 0, LIN_GLU = 1, LIN_SOFTCAP = 2, LIN_SCALE = 3, LIN_XIELU = 4, LIN_TANH_F = 5 };
struct LinArgs {
  const uint16_t* w;      // fragments
  const void* a_t;        // [rows][lda]
  int lda, kt, rt, rows;  // rt: row tiles that hold features
  int epi;                // LIN_*
  int n_wide;             // features below it go to out_t, the others (minus n_wide) to out_f (LIN_STORE); a multiple of 16
  void* out_t;
  int ld_t;
  float* out_f;
  int ld_f;
  float p0, p1, p2;       // LIN_GLU: limit, alpha, offset: min(g, limit) * sigmoid(alpha * g) * (clamp(u, +-limit) + offset); LIN_SOFTCAP: the cap;
                          // LIN_SCALE: the factor; LIN_XIELU: z > 0: p0 z^2 + z / 2, else p1 (exp(z) - 1 - z) + z / 2; LIN_TANH_F: tanh of the 32-bit part
  int a_seg, a_ops;       // a_seg > 0: features [i a_seg, (i + 1) a_seg) read operand i (the last one: the rest) of a_ops ...
  size_t a_stride;        // ... a_stride elements behind each other (launch_lin: a_seg is a multiple of 128, else of 16)
  int parts;              // > 1: k in `parts` ranges, each with a 32-bit output of its own (part_stride elements behind each other; n_wide = 0,
  size_t part_stride;     // LIN_STORE); the reader adds them up
  int tile;               // launch_lin: 0 chooses, 128 or 256 (bf16)
  const int* row_seq;     // launch_lin_few: output row i reads the first row of sequence row_seq[i] of seqs (nullptr: row i)
  const SeqDesc* seqs;
};
// parts worth splitting k into, at most `most`: launch_lin, launch_lin_few
int lin_parts(int rows, int rt, int kt, bool f32, int most);
int lin_parts_few(int rt, int kt, int most);
int launch_lin(hipStream_t st, const LinArgs& a, bool f32);          // any number of rows (tiles of 128)
int launch_lin_few(hipStream_t st, const LinArgs* a, int n, bool f32);  // up to 16 rows; n <= 4 products in one launch

// ---- experts ----
struct ExpertMat {          // one of the two matrices of a set of experts
  const uint16_t* w;        // routed experts, `stride` elements apart
  const uint16_t* shared;   // the shared expert's (nullptr: none)
  size_t stride;
  int kt, rt, shared_kt, shared_rt;
};
struct MoeArgs {
  int rows, width_ld, experts, top, shared;  // shared: 0 or 1 extra slot per row
  const float* logits;      // router logits [rows][ld_logits]
  int ld_logits;
  float* weight;            // [rows][top + shared]
  int* slot_pos;            // [rows][top + shared]: where the slot's hidden / output row is
  int* chosen;              // [rows][top]
  // many rows: slots sorted by expert
  int* count;               // [experts]
  int* cursor;              // [experts]
  int* slot_row;            // [rows * (top + shared)]: the row a sorted slot belongs to
  int* tiles;               // [max_tiles][4]: expert (experts = the shared one), first slot, slots, -
  int* n_tiles;
  int max_tiles;
  // few rows: the experts that any row chose
  int* active;              // [max_active]
  int* active_slot;         // [max_active][16]: slot (k) of each row, -1: not chosen
  int* n_active;
  int max_active;
  const void* h_t;          // the experts' input [rows][width_ld]
  void* hidden_t;           // [slots][hidden_ld]
  int hidden_ld;
  void* y_t;                // [slots][y_ld]
  int y_ld;
  ExpertMat up, down;
  float limit, shared_limit, alpha, offset;
};
enum { MOE_TILE = 128 };
int launch_route(hipStream_t st, const MoeArgs& a);                  // many rows: choose, sort
int launch_route_few(hipStream_t st, const MoeArgs& a);              // up to 16 rows
int launch_experts(hipStream_t st, const MoeArgs& a, bool down, bool f32);
// up to 16 rows; `also`: n_also plain products that ride in the same launch
int launch_experts_few(hipStream_t st, const MoeArgs& a, bool down, const LinArgs* also, int n_also, bool f32);

// ---- around the layers: residual sum, norms ----
// what a sandwich layer puts between a norm and its sublayer: h + a causal convolution of h, and blends with the previous token's
struct ConvArgs {
  int taps;
  const float* w;           // [width][taps], nullptr: no convolution
  size_t off_in;            // in the arena: the last taps - 1 inputs [2][taps - 1][width]
  const float* mu;          // [n_mix][width]: output i is y + (previous y - y) mu_i; nullptr: y alone
  int n_mix;
  size_t off_prev;          // the previous token's y [2][width]
  void* out_t;              // [n_mix or 1][rows][ld], mix_stride elements from blend to blend
  int ld;
  size_t mix_stride;
};
struct JoinArgs {           // x += (what the previous layer left); h = norm(x)
  PassDesc p;
  int width, h_ld;
  float eps, norm_offset;   // the norm's weight counts as w + norm_offset
  float* x;                 // [rows][width]
  const uint16_t* embed;    // first layer: x = embed[token] (nothing to add)
  const float* mix_a;       // mixer output [rows][mix_ld] (nullptr: none)
  int parts_a, parts_b;     // mix_a (mix_b) is the sum of this many, mix_stride elements behind each other
  size_t mix_stride;
  const float* mix_b;       // second of a pair: half the sum of both, each RMS-normed with its weight
  int mix_ld;
  const float *pair_wa, *pair_wb;
  const float* post_w;      // mix_a RMS-normed with this weight (+ norm_offset) first
  const void* y_t;          // expert outputs (nullptr: no feed-forward)
  int y_ld, n_slots;
  const int* slot_pos;
  const float* weight;
  const float* norm_w;      // nullptr: no norm, h is not written
  void* h_t;                // [rows or n_want][h_ld]
  int only_want;            // run the wanted rows only, h compact in their order (x is not written back)
  float* h_f;               // 32-bit h [rows][width] instead of h_t, for launch_conv
  ConvArgs conv;            // conv.w: single tokens, convolution and blends in the same launch (h_t and h_f are not used)
};
int launch_join(hipStream_t st, const JoinArgs& a, bool f32);
int launch_conv(hipStream_t st, const PassDesc& p, int width, const float* h_f, const ConvArgs& a, bool f32);

// ---- chunked softmax attention ----
struct ChunkAttnArgs {
  PassDesc p;
  int heads, kv_heads, dim, vdim, dim_p, vdim_p;  // *_p: padded to 32
  int chunk;
  float scale, eps;
  const void* proj_t;       // projections [rows][ld]; q, k, v start at these columns
  int ld, col_q, col_k, col_v;
  const float* freq;        // [rot_dims / 2]
  int rot_dims;
  float rot_amp;
  void *q_t, *k_t, *v_t;    // [rows][heads or kv_heads][*_p], filled by launch_chunk_prep
  size_t off_k, off_v;      // the layer's cache inside a sequence's arena: [chunk][kv_heads][*_p]
  void* out_t;              // [rows][out_ld]
  int out_ld;
};
int launch_chunk_prep(hipStream_t st, const ChunkAttnArgs& a, bool f32);
int launch_chunk_attn(hipStream_t st, const ChunkAttnArgs& a, bool f32);
int launch_chunk_store(hipStream_t st, const ChunkAttnArgs& a, bool f32);  // the last chunk's rows into the cache

// ---- recurrent mixers ----
enum { RECUR_MAX_DIM = 256, RECUR_CHUNK = 16 };
// A recurrence over chunks of 16 tokens as matrix products (kernels_chunk_scan.hip).  Per (chunk, head), in floats: the operands
// Kg [16][dim_p], Qg [16][dim_p], Ke [dim_p][16], Gend [dim_p], T [16][16], B [16][16]; dim_p = dim padded to 16.
static inline size_t chunk_floats(int dim) { return (size_t)49 * ((dim + 15) / 16 * 16) + 512; }
struct ChunkScan {
  float* ops;        // [n_chunks][heads][chunk_floats]
  float *keep, *add, *floor;  // mLSTM: [rows][heads] factors of the running maximum
};
struct DeltaArgs {          // gated delta rule with a decay per key channel, or one per head
  PassDesc p;
  int heads, kv_heads, dim, vdim, taps;
  float unit_eps, q_scale, eps;
  const void* proj_t;       // [rows][ld]
  int ld, col_q, col_k, col_v;
  const float* gate_f;      // beta logits [rows][ld_gate] from column col_b
  int ld_gate, col_b;
  const float* low_f;       // low-rank outputs [rows][ld_low]: decay input heads x dim, then the output gate heads x vdim
  int ld_low;
  int head_decay, col_a;    // one decay per head from gate_f; g is [rows][heads], dt_bias [heads]
  int silu_gate, col_g;     // silu of the projections' columns instead of the low-rank gate
  const float *conv_w;      // [channels][taps]: q, k, v channels behind each other
  const float *a_rate;      // [heads] exp(A_log)
  const float *dt_bias;     // [heads * dim]
  const float *out_norm;    // [vdim]
  float *q, *k, *v, *g, *beta;  // prepared inputs, [rows][...]
  float* o;                 // [rows][heads * vdim]
  size_t off_s, off_conv;   // state [heads][dim][vdim]; conv inputs [2][taps - 1][channels]
  void* out_t;
  int out_ld;
};
int launch_delta_prep(hipStream_t st, const DeltaArgs& a, bool f32);
int launch_delta_scan(hipStream_t st, const DeltaArgs& a);
int launch_delta_chunks(hipStream_t st, const DeltaArgs& a, const ChunkScan& c);  // instead of launch_delta_scan
int launch_delta_out(hipStream_t st, const DeltaArgs& a, bool f32);

struct MlstmArgs {          // matrix memory with exponential gates and a running maximum
  PassDesc p;
  int heads, dim, vdim;
  float q_scale, gate_cap, floor_eps, eps;
  const void* proj_t;
  int ld, col_q, col_k, col_v, col_g;
  const float* gate_f;      // input / forget gate logits
  int ld_gate, col_i, col_f;
  const float *b_i, *b_f, *out_norm;
  float* o;
  size_t off_s, off_n, off_m;  // [heads][dim][vdim], [2][heads][dim], [2][heads]
  void* out_t;
  int out_ld;
};
int launch_mlstm_scan(hipStream_t st, const MlstmArgs& a, bool f32);
// ... instead of launch_mlstm_scan: o gets vdim + 1 columns per head, the sums before the division and the normaliser behind them
int launch_mlstm_chunks(hipStream_t st, const MlstmArgs& a, const ChunkScan& c, bool f32);
int launch_mlstm_out(hipStream_t st, const MlstmArgs& a, const ChunkScan* c, bool f32);  // c: o comes from launch_mlstm_chunks

struct WkvArgs {            // S <- diag(w) S + k v^T, read before it with a bonus u for the current token
  PassDesc p;
  int heads, dim;
  float eps;
  const void* proj_t;       // r, k, v and the gate
  int ld, col_r, col_k, col_v, col_g;
  const float* low_f;       // second half of the decay's low-rank pair [rows][ld_low]: w = exp(-exp(low + w0))
  int ld_low;
  const float *w0, *u, *out_norm;  // [heads * dim]
  float* o;
  size_t off_s;             // [heads][dim][dim]
  void* out_t;
  int out_ld;
};
int launch_wkv_scan(hipStream_t st, const WkvArgs& a, bool f32);
int launch_wkv_chunks(hipStream_t st, const WkvArgs& a, const ChunkScan& c, bool f32);  // instead of launch_wkv_scan
int launch_wkv_out(hipStream_t st, const WkvArgs& a, bool f32);

// ---- latent attention in a sliding window (kernels_latent.hip) ----
// A token leaves one latent row [rank_p + rot_p]: the normed latent, then the rotated key part.  The cache is a ring of `window` latent
// rows (row = position % window).  Portions of several tokens expand the rows they see to keys and values per head; single tokens
// carry their query into the latent space instead and read the ring as it is.
struct LatentArgs {
  PassDesc p;
  int heads, dim, rot_dim, vdim, q_rank, kv_rank, window, rot_dims;
  int dim_p, rot_p, vdim_p, rank_p;  // padded to 32, 32, 32, 64
  float scale, eps;
  const float* proj_f;      // 32-bit projections [rows][ld]: query latent, then [latent, rotated key part]
  int ld, col_q, col_kv;
  const float *q_norm, *kv_norm, *freq;
  void* cq_t;               // normed query latents [rows][cq_ld], zero up to a multiple of 64 columns
  int cq_ld;
  float* turn;              // cosines, then sines of a row's angles [rows][rot_dims]
  void* q_t;                // queries [rows][q_ld], per head [dim_p][rot_p], not rotated yet
  int q_ld;
  void* lat_t;              // key workspace: latent rows [key rows][rank_p + rot_p]
  const void* kv_t;         // ... expanded [key rows][heads * dim_p + heads * vdim_p]
  int kv_ld;
  size_t off_c;             // the ring in a sequence's arena
  void* out_t;              // [rows][out_ld]
  int out_ld;
  // single tokens, up to 16 at a time: sequences p.single[first .. first + n)
  int first, n, splits;     // workgroups per token, latent_keys() keys each: enough for the longest
  const void* qa_t;         // queries in the latent space [16][heads * rank_p]
  float *part, *part_ml;    // [16][heads][splits][rank_p], [...][2]
  const uint16_t* up_w;     // fragments of the expansion (the value half is used): row of head h, value 0 is up_row + h * vdim_p
  int up_kt, up_row;
};
int latent_keys(bool f32);
int launch_latent_prep(hipStream_t st, const LatentArgs& a, bool f32);    // norms, rotation; single tokens' rows go into their rings
int launch_latent_gather(hipStream_t st, const LatentArgs& a, bool f32);  // older rows from the rings into the key workspace
int launch_latent_turn(hipStream_t st, const LatentArgs& a, bool f32);    // rotates the queries of portions of several tokens
int launch_latent_attn(hipStream_t st, const LatentArgs& a, bool f32);    // portions of several tokens
int launch_latent_store(hipStream_t st, const LatentArgs& a, bool f32);   // their rows into the rings
int launch_latent_few(hipStream_t st, const LatentArgs& a, bool f32);     // single tokens: scores, weights, latent sums, values

// ---- steps of up to 16 single tokens: everything between a layer's projection and its output products in one launch ----
struct MixFewArgs {
  int rows;                   // one token of `rows` sequences
  int has_attn, has_mlstm, has_delta, has_wkv, has_route;
  ChunkAttnArgs attn;         // (q_t, k_t, v_t are not used: rotation and norms happen inside)
  int splits;                 // workgroups per (sequence, key head), ATTN_SPLIT_KEYS keys each: enough for the longest
  float* part;                // [rows][heads][splits][vdim_p + 2]
  unsigned* arrived;          // [rows][kv_heads], zero between launches
  MlstmArgs mlstm;
  DeltaArgs delta;            // (q, k, v, g, beta, o are not used)
  const uint16_t* low_w;      // the low-rank second halves (fragments, block-diagonal): low_a input columns, then low_g
  int low_kt, low_a, low_g;
  int col_low;                // their inputs' column in proj_t
  WkvArgs wkv;                // (o is not used)
  const float* wkv_low;       // the decay's low-rank first half [rows][wkv_low_ld], 32-bit; its second half is low_w with low_a columns
  int wkv_low_ld;
  MoeArgs moe;
};
enum { ATTN_SPLIT_KEYS = 128 };
bool mix_few_fits(const MixFewArgs& a);
int launch_mix_few(hipStream_t st, const MixFewArgs& a, bool f32);
