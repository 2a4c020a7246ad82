// engine.h -- the host runtime's state behind the C ABI (mi_engine, mi_kv) and the helpers that its translation units share:
// engine.hip (the ABI, uniform decoder stacks, cache management, sampling) and engine_layers.hip (layer-list models).
#pragma once
#include <algorithm>
#include <cstring>
#include <list>
#include <map>
#include <string>
#include <unordered_map>
#include <vector>

#include "kernels.h"

namespace mi {

struct FusedLinear {
  LinearW W;
  int parts = 0;                 // bit mask of sub-tensors seen (weight / scales / biases per part)
  int n_parts = 1;
  int part_rows[3] = {0, 0, 0};
  bool quant = false;
  int dense_dtype = -1, scale_dtype = -1;
  size_t w_bytes = 0, s_bytes = 0;
  void* w = nullptr; void* scales = nullptr; void* biases = nullptr;
  // Persistent second copies of a matrix (made by mi_engine_finalize, i.e. BEFORE a scheduler sizes its KV arena from the
  // free device memory; a pointer is published only after its repack launch succeeded; when the allocation fails the
  // copy is marked unavailable and the linear keeps its plain path -- ensure_hilo / ensure_gu8)
  void* w_hilo = nullptr;        // f16 dense weights in the float32-activation (PagedKVCache) mode: [hi | lo] bf16 copy
  void* w_gu8 = nullptr;         // dense 16-bit gate|up: row-interleaved copy for the decode GEMV (EPI_SWIGLU_GU8)
  bool hilo_failed = false, gu8_failed = false;
  float* lora_a[2] = {nullptr, nullptr};
  float* lora_b[2] = {nullptr, nullptr};
  int seen_w[3] = {0, 0, 0}, seen_s[3] = {0, 0, 0}, seen_b[3] = {0, 0, 0};
};

struct LayerW {
  FusedLinear qkv, o, gate_up, down;
  void* in_norm = nullptr; void* post_norm = nullptr; void* q_norm = nullptr; void* k_norm = nullptr;
  // float32 copies for the float32-activation ("PagedKVCache quirk") mode
  void* in_norm32 = nullptr; void* post_norm32 = nullptr; void* q_norm32 = nullptr; void* k_norm32 = nullptr;
};

// A matrix assembled from several checkpoint tensors: each part is a rectangle of the zero-filled [N][K] buffer (rows AND
// columns may be padded), so that several projections of one input run as one launch (parts stacked along N) and several
// outputs that are summed run as one launch (parts side by side along K).
struct PackedPart { std::string name; int row0, col0, rows, cols; bool seen; };
struct PackedLinear {
  FusedLinear f;
  int N = 0, K = 0;
  std::vector<PackedPart> parts;
};

// A small tensor kept in float32 whatever the model dtype (norm weights, decay parameters, convolution taps)
struct Vec32 { std::string name; int n = 0; float* p = nullptr; bool seen = false; bool optional = false; float add = 0.f; };   // add: on top of what is stored

// One layer of a layer-list model
struct ListLayer {
  mi_layer_desc d{};
  PackedLinear in, out;          // every projection of the normed input; [mixer output | activation] -> residual
  // element offsets of the parts in a row of `in`'s output, and of the activation in a row of `out`'s input
  int o_q = -1, o_k = -1, o_v = -1, o_g = -1, o_b = -1, o_a = -1, o_c = -1, o_up = -1, o_ff = 0;
  int n_cat = 0;                 // columns of `out`'s input
  Vec32 norm, act;
  // delta rule
  Vec32 conv_q, conv_k, conv_v, A_log, dt_bias, head_norm;
  // low-rank maps: the inner projections (decay | gate) lie side by side in `in`'s output from o_lr, the outer ones are one matrix
  // over both (block-diagonal); o_a / o_g then count in a row of its output
  PackedLinear lr;
  int o_lr = -1, o_lrg = -1;     // (o_lrg: the gate's)
  void* low_a = nullptr; void* low_g = nullptr;      // the outer maps row-major (one-token segments), stride a multiple of 8
  // latent attention
  Vec32 c_norm;
  PackedLinear uq;               // queries from their latent
  Vec32 dq_norm;
  int o_qc = -1, qr = 0, cp = 0; // the queries' latent in a row of `in`'s output, its padded size; place of the rotated key part in a cached row
  PackedLinear ukv;              // [heads x kdp key rows | heads x vdp value rows] over the latent (padded per head)
  void* uk = nullptr; void* uv = nullptr;    // the two maps as loaded, [heads * dim][kv_rank] / [heads * vdim][kv_rank]
  void* uk_t = nullptr;          // [heads][latent (padded)][kdp]: the key map transposed, for queries absorbed into the latent space
  void* uv_p = nullptr;          // [heads][vdim][latent (padded)]
  bool uk_seen = false, uv_seen = false;
  int kdp = 0, vdp = 0, rp = 0;  // padded key / value / latent sizes
  int src = -1;                  // the layer whose latents this layer reads (itself or kv_from)
  // per-layer token input
  void* side_gate = nullptr; void* side_proj_t = nullptr; void* side_proj_p = nullptr;   // [dim][width], transposed [dim][width], padded [width][dim]
  bool side_gate_seen = false, side_proj_seen = false;
  Vec32 side_norm;
  // grouped-query attention (q_norm, k_norm: ones where the norm has no weights)
  Vec32 q_norm, k_norm, vmix, sink;
  const float2* rot_tab = nullptr;   // owned by the engine (mi_engine::rot_tabs)
  float* slopes = nullptr;       // [heads] distance bias
  bool v_first = false;          // the first layer whose values are mixed: the later ones read its values
  bool gqa_fast = false;         // matrix-core forms
  float rot_gain = 1.f;
  // lightning attention (its norm: head_norm)
  float* decay = nullptr; float* log2_decay = nullptr;      // [heads]
  int sd = 0;                    // row stride of the state
  // `norm` is in front of a parallel block and of a pre-norm or sandwich mixer, behind a post-norm one; norm2 the feed-forward's; norm_out,
  // norm2_out: behind the sublayers of a sandwich block
  Vec32 norm_b, norm2, norm2_b, norm_out, norm2_out;
  // hyper-connections of the two sublayers: weights of the streams in what is read, [from][to], of the output in the streams
  Vec32 hc_in[2], hc_mix[2], hc_out[2];
  // SwiGLU feed-forward: gate | up and down matrices (gu, dn); mixture of experts: all routed experts' stacked, the shared expert's
  PackedLinear gu, dn, sgu, sdn;
  int ffp = 0, sffp = 0;         // padded widths
  void* router = nullptr;        // [experts][padded width] row-major
  bool router_seen = false;
  Vec32 router_b;
  Glu glu;                       // the feed-forward's unit
};

// One pass through a layer: what it keeps between calls is its own, also where a layer runs more than once
struct LayerRun { int layer; int lat = -1, k = -1, v = -1, state = -1; };      // arenas of the latents, keys, values; recurrent-state slot

// one slab of the cache of a layer-list model: [place][heads][width] elements per token from element offset `off`
struct KvArena { size_t off; int heads, width; };

constexpr int NSLOT = 4;
struct Slot {
  hipEvent_t ev = nullptr;
  int32_t* tokens = nullptr; float* logprob = nullptr; float* prob0 = nullptr;
  int32_t* topk_ids = nullptr; float* topk_lp = nullptr;   // pinned host
  int B = 0, topk = 0; int64_t ticket = -1;
};

}  // namespace mi

using namespace mi;

struct mi_engine {
  mi_model_desc d{};
  int device = 0;
  hipStream_t stream = nullptr;
  std::vector<LayerW> layers;
  FusedLinear embed, lm_head;
  void* final_norm = nullptr; void* final_norm32 = nullptr;
  bool finalized = false;
  float* cos_tab = nullptr; float* sin_tab = nullptr;
  // workspace
  size_t ws_rows = 0; size_t ws_logit_rows = 0;
  void* h = nullptr; void* qkv = nullptr; void* q = nullptr; void* attn = nullptr; void* act = nullptr;
  float* logits = nullptr; float* lora_t = nullptr;
  int32_t* d_tokens = nullptr; size_t d_tokens_cap = 0;
  const int32_t* tok_src = nullptr;                       // device-fed step: the embedding reads the sampler's output in place
  int32_t* d_forced = nullptr; size_t d_forced_cap = 0;   // mi_score_tokens targets
  int32_t* d_gather = nullptr;                            // token positions whose hidden state feeds the head (mixed steps)
  float* d_rowpar = nullptr; size_t d_rowpar_cap = 0;     // per-row temperature | top_p of the current step
  void* deq_scratch = nullptr; size_t deq_cap = 0;        // [hi | lo] 16-bit copy of one int4 matrix (prefill GEMM)
  void* sk_ws = nullptr; size_t sk_ws_cap = 0;            // split-K partial tiles of gemm_skinny.hip
  unsigned* sk_ctr = nullptr; int sk_ctr_cap = 0;         // its per-tile-group arrival counters (zero between launches)
  int32_t* d_next = nullptr;      // tokens sampled by the last step [maxB]
  float* d_logprob = nullptr; float* d_prob0 = nullptr; float* d_rowstats = nullptr; float* d_uniforms = nullptr;
  int32_t* d_topk_ids = nullptr; float* d_topk_lp = nullptr;
  int32_t* d_bias_ids = nullptr; float* d_bias_vals = nullptr;
  int maxB = 0;
  int max_lora_rank = 0;
  Slot slots[NSLOT];
  int64_t next_ticket = 0;
  uint64_t step_counter = 0;
  // profiling
  std::string prof_name;
  std::vector<std::pair<hipEvent_t, hipEvent_t>> prof_events;
  int opt_force_v1 = 0;
  int opt_fused_attn = 1;
  int opt_attn_mfma = 1;                 // decode attention on the matrix cores where the shape allows
  int opt_tile_weights = 1;
  int opt_prefill_gemm = 1;
  int opt_skinny_gemm = 1;      // decode steps of 9..128 rows (int4 / int8: 1..128): the split-K weight-streaming GEMM (gemm_skinny.hip)
  int cur_L = 0;                // tokens per sequence of the forward pass being enqueued
  // RMSNorm hand-over between gemm_skinny launches (GemvCall::sq_out / sq_in): the residual linear in front of a norm
  // leaves the rows' sums of squares, the normalised linear behind it uses them instead of an rmsnorm launch
  int opt_norm_handover = 1;    // round 2 (partial sums read in ONE round trip): Mistral-7B int4 +3.2 %, int8 +2.9 %, bf16 B = 16 +3.7 %, Qwen3-14B int4 +0.6 %
  int opt_prefill_x_terms = 2;  // float32 activations, prefill tile GEMM on dense bf16 weights: 16-bit terms of x (2 or 3 = exact)
  int opt_defer_norm = 1;       // float32 activations: RMSNorm row scale applied in the split-K kernel's epilogue (no norm launch)
  int opt_short_prefill_skinny = 1;   // short prefill / mixed calls on the weight-streaming kernel instead of the tile GEMM (gemv_rows)
  float* d_sq = nullptr;        // [4096 tile groups][16 rows]
  bool sq_valid = false; const void* sq_src = nullptr; int sq_parts = 0, sq_K = 0, sq_ld = 0;
  bool opt_gu8 = true;                   // decode GEMV of a dense gate|up matrix on its row-interleaved copy: 7 one-tile items per CU instead of 3.5 pairs (twice the matrix's bytes)
  bool opt_f16_hilo = true;              // f16 dense weights in the float32-activation mode through an exact [hi | lo] bf16 copy (matrix cores)
  int opt_fused_pairs = 0;               // bit 0: o_proj -> gate|up, bit 1: down_proj -> next q|k|v as one launch each.
                                         // Off: measured on Mistral-7B bf16 B=8 the in-launch seam costs what the kernel
                                         // boundary it replaces costs (bit 0: +-0 %, bit 1: -2 %), DESIGN.md section 5
  unsigned* d_seam_counter = nullptr;    // arrival counter of the in-launch seams (monotonic)
  int* d_seam_error = nullptr;           // set by a workgroup that gave up waiting at a seam
  int* h_seam_err = nullptr;             // pinned: [slot] = *d_seam_error behind that step's launches, [NSLOT] = synchronous reads
  unsigned seam_spin_limit = 1u << 20;   // polls before a workgroup gives up (option "seam_spin_limit"; tests force 0)
  unsigned seam_base = 0;
  int last_n = 0;                        // rows of the last enqueued step (device-resident token feed)                // value of *d_seam_counter once every enqueued launch has run
  void* xn = nullptr;            // [rows][max(H, I)] normalised activations of the prefill GEMMs
  void* xs = nullptr; size_t xs_cap = 0;   // [rows][3 K] bf16: float32 activations split three ways (float32-KV prefill)
  void* gk_ws = nullptr; size_t gk_cap = 0;   // float32 partial tiles of the K-split 128 x 128 tile GEMM
  // ---- layer-list models (engine_layers.hip)
  bool layered = false;
  std::vector<ListLayer> list;
  std::vector<LayerRun> runs;    // the layers in the order in which they run
  int n_arena = 0, n_state = 0;
  struct RotTab { int dims; float base, factor, original, fast, slow, gain; float2* p; };
  std::vector<RotTab> rot_tabs;  // one per rotation
  int streams = 1;               // copies of the residual stream
  void* pair_embed = nullptr; bool pair_embed_seen = false;   // [pair_buckets + 1][width]
  void* low = nullptr;           // [rows][max N of `lr`]
  float* dl_q = nullptr; size_t dl_q_cap = 0;                 // channel form: queries with their decays
  void* qc = nullptr; void* qfull = nullptr;                  // latent attention: [rows][max qr] queries' latents, [rows][max uq.N] queries
  bool any_light = false, any_latent = false;
  int latent_qt = 128;           // queries per tile of the latent attention's longer portions, at most
  float* light_ws = nullptr; size_t light_ws_cap = 0;         // lightning attention: matrices of the chunks
  int* light_ctr = nullptr; size_t light_ctr_cap = 0;         // arrival tickets of its one-token form (zero between launches)
  PackedLinear list_head;
  Vec32 list_final_norm, list_final_norm_b;
  float* y32 = nullptr;          // [rows][wp] a sublayer's output in front of its norm / of the residual update
  int n_vfirst = 0;
  void* v_first = nullptr;       // [rows][n_vfirst] values of the first mixing layer
  int32_t* moe_ids = nullptr; float* moe_wts = nullptr;       // [rows][max top]
  void* moe_mid = nullptr; void* moe_out = nullptr;           // [slots][max ff], [slots][wp]
  int32_t* moe_plan = nullptr; int32_t* moe_counts = nullptr;
  int gqa_chunk = -1, gqa_window = 0;      // of the first grouped-query layer (order of the query tiles); -1: no such layer
  float* gqa_part = nullptr; size_t gqa_part_cap = 0;         // split-KV partials of the decode attention
  int* gqa_ctr = nullptr; size_t gqa_ctr_cap = 0;             // its arrival tickets (zero between launches)
  void* tok_embed = nullptr; bool tok_embed_seen = false;     // [vocab][width] row-major
  void* side_embed = nullptr; bool side_embed_seen = false;   // [vocab][layers * side_dim]
  double* d_freq = nullptr;      // [ceil(width / 2)] angular frequencies of the sinusoidal positions
  int wp = 0;                    // padded width: row stride of the residual stream and of the normed input
  size_t lw_rows = 0;            // workspace rows
  float* x32 = nullptr;          // [rows][streams][wp] residual stream
  void* hn = nullptr;            // [rows][wp] normed input (model dtype)
  void* proj = nullptr;          // [rows][max N of `in`]
  void* cat = nullptr;           // [rows][max K of `out`]
  float* scan32 = nullptr;       // [rows][max q | k | v floats] inputs of the recurrence, its outputs in place of v
  float* gate32 = nullptr;       // [rows][max heads][4] decay, step size, k . q
  void* lq = nullptr;            // [rows][max heads * padded latent] queries in the latent space
  float* lat_part = nullptr; size_t lat_part_cap = 0;         // split-KV partials of the latent decode attention
  void* lat_x = nullptr; size_t lat_x_cap = 0;                // gathered latents of a prefill call [keys][padded latent]
  void* lat_m = nullptr; size_t lat_m_cap = 0;                // decode: the splits merged
  float* dl_w = nullptr; size_t dl_w_cap = 0;                 // chunked delta rule: what delta_chunk leaves for delta_carry
  float* dl_p = nullptr; size_t dl_p_cap = 0;
  float* dl_k = nullptr; size_t dl_k_cap = 0;
  float* dl_f = nullptr; size_t dl_f_cap = 0;
  void* lat_kv = nullptr; size_t lat_kv_cap = 0;              // their keys | values
  int32_t* d_meta = nullptr; size_t d_meta_cap = 0;           // segment / tile tables of the current call
  std::vector<int32_t> h_meta;
  int scan_ld = 0, gate_ld = 0;
  int32_t* d_gather_list = nullptr; size_t d_gather_list_cap = 0;   // wanted positions, their normed rows
  void* head_x = nullptr; size_t head_x_cap = 0;
  float* resid_out = nullptr; int64_t resid_cap = 0;          // mi_debug_residual
};


struct mi_kv {
  mi_engine* e = nullptr;
  int B = 0, cap = 0, dtype = MI_F32;
  bool quirk = false;            // float32 "PagedKVCache" semantics on a 16-bit model
  void* k = nullptr; void* v = nullptr;
  int32_t* d_off = nullptr;
  std::vector<int32_t> h_off;
  int32_t* d_rows = nullptr;     // [B] scratch: cache rows of the current call (continuous batching)
  float* partial = nullptr; int partial_splits = 0;
  int* counters = nullptr;       // [B*Hkv] split-arrival tickets of the fused decode attention
  // ---- block-paged form (mi_kv_create_paged): k / v are arenas [layer][block][Hkv][1 << bs_shift][D]; a row owns the
  // blocks its table names, in order; block 0 is never handed out (unassigned table entries point at it, so a clamped
  // address is always mapped memory); cap = bt_stride << bs_shift is the longest sequence a row can hold
  bool paged = false;
  int bs_shift = 0, nblocks = 0, bt_stride = 0;
  int32_t* d_btab = nullptr;
  std::vector<int32_t> h_btab;   // [B][bt_stride]
  std::vector<int> row_blocks;   // blocks in use per row
  std::vector<int> refcnt;       // per block: rows that map it + 1 if the prefix cache holds it
  std::vector<int> free_blocks;
  bool btab_dirty = false;
  // prefix cache: full blocks of prompts, keyed by the hash of ALL tokens up to and including the block; an entry keeps
  // the block's own tokens and its parent's key, so a hit is verified token by token (no reliance on the hash alone)
  struct PrefixEntry { int block; uint64_t parent; std::vector<int32_t> tokens; std::list<uint64_t>::iterator lru_it; };
  std::unordered_map<uint64_t, PrefixEntry> prefix;
  std::list<uint64_t> lru;       // front = most recently used
  int64_t stat_hit_tokens = 0, stat_lookup_tokens = 0, stat_evictions = 0;
  // ---- layer-list models: latents, keys and values live in k (one arena per layer that has its own latents, two per
  // grouped-query layer; the same block table for all), recurrent layers in `state` (one slot per cache row)
  std::vector<KvArena> arenas;
  char* state = nullptr;
  size_t list_bytes = 0, state_bytes = 0;
  std::vector<size_t> state_off, ring_off;   // bytes: [row][heads][dim][vdim] float32 (lightning: [row][heads][vdim][sd]), [row][taps][channels] model dtype
  int32_t* d_prev = nullptr;     // [row] last token (inside `state`; a model whose embedding looks at the previous token)
};

namespace mi {

struct Prof {
  mi_engine* e; bool on; hipEvent_t a = nullptr, b = nullptr;
  Prof(mi_engine* e_, const char* name) : e(e_), on(!e_->prof_name.empty() && e_->prof_name == name) {
    if (on) { hipEventCreate(&a); hipEventCreate(&b); hipEventRecord(a, e->stream); }
  }
  ~Prof() { if (on) { hipEventRecord(b, e->stream); e->prof_events.emplace_back(a, b); } }
};

int copy_in(void* dst, const void* src, size_t bytes, int on_device, hipStream_t st);
int finalize_linear(mi_engine* e, FusedLinear& f, int K, const std::string& name);
void free_linear(FusedLinear& f);
bool ensure_gu8(mi_engine* e, FusedLinear& f, int pair_offset);
// y = W x for `rows` rows on the kernel family that fits the call; es_in / es_out: element sizes of x and out
int gemv_rows(mi_engine* e, const FusedLinear& f, GemvCall c, size_t rows, size_t es_in, size_t es_out, const char* prof);
int kv_ensure_blocks(mi_kv* kv, int row, int tokens);
int kv_upload_table(mi_kv* kv, hipStream_t st);
void kv_shape(const mi_kv* kv, AttnShape& s);

// ---- layer-list models (engine_layers.hip)
int layers_set_tensor(mi_engine* e, const std::string& name, const void* data, const int64_t* shape, int ndim, int dtype, int on_device);
int layers_finalize(mi_engine* e);
void layers_free(mi_engine* e);
int layers_kv_plan(mi_engine* e, mi_kv* kv);                 // arena layout + recurrent-state buffers of a new cache
void layers_kv_bind(mi_engine* e, mi_kv* kv);               // pointers into the allocated state
int layers_ensure_workspace(mi_engine* e, size_t rows);
// segment i = lens[i] tokens of cache row rows[i]; tokens (the concatenation) already on the device; logits of the token
// positions out_idx[0..n_out) end up in e->logits [n_out][vocab]
int forward_segments(mi_engine* e, mi_kv* kv, const int32_t* rows, const int32_t* lens, int n, const int32_t* out_idx, int n_out);

}  // namespace mi
