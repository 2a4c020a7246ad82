// layer_kernels.h -- host-side launch interface of the kernels of layer-list models (internal to the library).
#pragma once
#include "kernels.h"

namespace mi {

// ---- layer-list models: a call covers n segments (segment = tokens of one cache row), R tokens in all -----------------------
constexpr int DELTA_CHUNK = 64;  // tokens the chunked form of the delta rule takes at a time
constexpr int DELTA_FAC = 2 * DELTA_CHUNK + 4;   // per chunk and value head: factors of q, of X in the state, and of the state
struct SegTables {               // device tables of one call (engine_layers.hip: build_tables)
  const int32_t* row;            // [n] cache row of the segment
  const int32_t* tok0;           // [n] its first token
  const int32_t* len;            // [n]
  const int32_t* kbase;          // [n] its first row among the gathered keys (prefill segments)
  const int32_t* cbase;          // [n] its first chunk in ctile (prefill segments)
  const int32_t* tok_seg;        // [R] segment of a token
  const int32_t* dec;            // [nd] one-token segments
  const int32_t* chunk;          // [nc] segments of two tokens and more
  const int32_t* tile;           // [nt][2] query tiles of the chunks: segment, first token in the segment
  const int32_t* gtile;          // [ngt][2] key tiles of the chunks: segment, first key
  const int32_t* ctile;          // [nct][2] whole chunks of DELTA_CHUNK tokens of the chunk segments: segment, first token
  const int32_t* off;            // [cache rows] tokens in the cache before this call (mi_kv::d_off)
  int n, R, nd, nc, nt, ngt, nct;
  int qt;                        // queries per query tile: 64 or 128
};

struct RowNormW { const float* w; int stride; float eps; };     // stride 1: a weight per coordinate, 0: one number for all

// x = scale table[token] (+ sinusoidal position) (+ a row of the table of token pairs), h = norm(x) (norm.w null: h = x) in the
// activation dtype; columns [width, ld) are zero.  With several streams every one of them is x, and h = norm(sum_s in[s] x).
// (layer_rows.hip)
struct PairEmbed { const void* table; int buckets, mul_prev, mul_cur; const int32_t* prev; };   // table [buckets + 1][width] or null; prev
                                 // [cache rows]: a row's last token before this call.  Row (prev mul_prev + token mul_cur) mod buckets,
                                 // the last one for the first token of a sequence
struct EmbedPosCall {
  SegTables t;
  const int32_t* tokens;
  const void* table;             // [vocab][width] row-major
  const double* freq;            // [ceil(width / 2)] or null: no positions
  int vocab, width, ld;
  RowNormW norm;
  float* x; void* h;             // x [R][max(1, streams)][ld]
  int act;
  float scale;
  PairEmbed pair;
  int streams; const float* in;  // streams 0: one plain stream, in is null
};
int launch_embed_pos(const EmbedPosCall& c, hipStream_t st);

// Per-layer token input + the norm in front of what follows:
//   x += rms(proj (gelu_tanh(gate x) * table[token][slice])) * side_w ;  h = norm(x)       (dim = 0: only the norm)
struct SideNormCall {
  int rows;
  const int32_t* tokens;
  const void* table; int table_ld, slice, vocab;   // [vocab][table_ld], the layer's columns [slice, slice + dim)
  const void* gate;              // [dim][ld] (columns beyond width are zero)
  const void* proj_t;            // [dim][ld]
  const void* proj_p;            // [ld][dim rounded up to 32] for the matrix-core form, or null
  const float* side_w; float side_eps;
  int dim, width, ld;
  RowNormW norm;
  float* x; void* h;
  int act;
};
bool side_mfma_supported(int act, int dim, int ld);
int launch_side_norm(const SideNormCall& c, hipStream_t st);

// off[row of each segment] += its length; prev (or null): the row's last token
int launch_advance_segments(const SegTables& t, int32_t* off, const int32_t* tokens, int32_t* prev, hipStream_t st);

// Residual update of a pre-norm block and the norm in front of what follows.  One stream (streams 0): x += mult y, h = norm(x).
// Several: x_t <- sum_s mix[s][t] x_s + mult out[t] y from the old ones, h = norm(sum_s in[s] x_s); in null: h = norm(sum_s x_s).
struct StreamNormCall {
  int rows;
  const float* y;                // [rows][ld] a sublayer's output
  int streams;
  const float* mix; const float* out; const float* in;
  float mult;
  RowNormW norm;
  int width, ld;
  float* x; void* h;             // x [rows][max(1, streams)][ld]
  int store;                     // 0: the streams are not needed any more
  int act;
};
constexpr int MAX_STREAMS = 16;
int launch_stream_norm(const StreamNormCall& c, hipStream_t st);
int launch_stream_sum(const float* x, int streams, int rows, int ld, float* out, hipStream_t st);     // out [rows][ld]
// tab [positions][pairs]: gain times cosine and sine of p freq[i] (angles in double precision); freq [pairs] on the device
int launch_rotation_table(float2* tab, int positions, int pairs, const double* freq, double gain, hipStream_t st);

struct PolyNormArgs { int ff, in_off, out_off; const float* coef; float eps; };     // ff = 0: none

// Gated delta rule (delta.hip).  Channels of the convolutions, their ring and the scan buffer: [q: G d | k: G d | v: H e], in the scan
// buffer of a rule with a decay per channel also [decays: H d]
struct DeltaCall {
  SegTables t;
  int H, G, d, e, taps;
  const void* proj; int ldp;     // [R][ldp] outputs of the fused input projection
  int o_q, o_k, o_v, o_b;
  const void* ap; int ldap, o_a; // [R][ldap] what the decays are made of: one per value head, or (channel) one per value head and key channel
  const void* gp; int ldgp, o_g; // [R][ldgp] output gates, [H e]
  int channel, gate_act;         // gate_act: MI_GATE_SILU or MI_GATE_SIGMOID
  // one-token segments make both from the inner projections themselves (null: from ap, gp): outer maps [H d][ld_a], [H e][ld_gt] (strides
  // padded with zeros to a multiple of 8), the inner projections' places in a row of proj
  const void* low_a; const void* low_g; int ld_a, ld_gt, in_a, in_g;
  const float* conv_q; const float* conv_k; const float* conv_v;    // [channels][taps]
  const float* A_log; const float* dt_bias; const float* head_norm;       // dt_bias [H] or (channel) [H d]
  float scale, unit_eps, eps;
  float* state;                  // [cache row][H][d][e]
  void* ring;                    // [cache row][taps][channels]: the inputs of position p at slot p mod taps
  float* scan; int lds;          // [R][lds] prefill: q, k, v in 32 bit; the outputs replace v
  float* gate; int ldg;          // [R][ldg] four numbers per value head: decay, step size, k . q (token by token)
  float* wm; float* pm;          // chunked form: [R][H][padded d], [R][H][DELTA_CHUNK]; null: token by token
  float* kt; float* fac;         // [chunks][G][padded d][DELTA_CHUNK] unit keys transposed, [chunks][H][DELTA_FAC]
  float* qm;                     // channel: [R][H][padded d] unit queries with their decay from the chunk's start; then kt is [chunks][H]..
                                 // (keys with their decay to the chunk's end) and fac [chunks][H][padded d] (the whole chunk's decay)
  void* cat; int ldc;            // [R][ldc] mixer output from column 0
  PolyNormArgs ff;
  int act;
};
int launch_delta(const DeltaCall& c, hipStream_t st);
bool delta_supported(int d, int e);
int delta_chunk_pad(int H, int d, int e, int taps);     // padded head size of the chunked form, 0 = not supported

// The outer low-rank maps of many rows (delta.hip): out[r][0 .. n) = W x[r], where rows [0, split) of W use the columns [0, k) of x and
// W, the rows behind them the next k (W is block-diagonal).  16-bit, tile-major W, split a multiple of 16.
struct LowRankCall { LinearW W; int split, k; const void* x; int ldx, rows; void* out; int ldo, act; };
bool low_rank_supported(const LowRankCall& c);
int launch_low_rank(const LowRankCall& c, hipStream_t st);

// Latent attention (latent.hip): the cache holds one latent per token, [token][rp]; keys and values are maps of it.  With a rotated part
// (rot > 0) a token's row is [latent | padding to cp | rotated key part, one for all heads | padding], a query head [dim | rot], and a
// score the sum of both products.
struct LatentCall {
  SegTables t;
  AttnShape s;                   // cache addressing: Hkv = 1, D = rp, cap / btab as usual
  int H, dim, vdim, rank, rp, kdp, vdp;
  int rot, cp, pairs; const float2* rot_tab;       // size of the rotated part (0: none), its place in a cached row, MI_ROT_*, [position][rot / 2]
  const void* proj; int ldp;
  int o_g, o_c;                  // o_g < 0: no gate; o_c < 0: the latents are another layer's, nothing is appended
  const void* q; int ldq;        // [R][ldq] queries, head h's dim + rot from element h (dim + rot) on
  int q_rank, ldqc; const float* q_norm; void* qc; int o_qc;      // q_rank > 0: latent_pre leaves rms(proj from o_qc on) * q_norm in qc [R][ldqc]
  const float* c_norm; float eps;
  void* cache;                   // the arena of the layer the latents belong to
  const void* uk; const void* uv;          // [H * dim][rank], [H * vdim][rank]
  const void* uk_t; const void* uv_p;      // [H][rp][kdp], [H * vdim][rp] (16-bit forms)
  float scale;
  void* lq;                      // [R][H][rp] queries in the latent space (generic form: float32)
  float* partial; int nsplit;    // decode: [nd][head tiles x 16][nsplit][rp + 4]
  void* merged;                  // decode: [nd][H][2][rp]
  const void* kv; int ldkv;      // prefill: keys | values of the gathered latents [keys][H kdp + H vdp]
  void* cat; int ldc;
  PolyNormArgs ff;
  int act;
};
int launch_latent_pre(const LatentCall& c, hipStream_t st);            // append the latents, feed-forward activation, the queries' latent
int launch_latent_generic(const LatentCall& c, hipStream_t st);        // any size and dtype, all tokens
int latent_tile(int kdp, int vdp);                                            // queries per tile at most
bool latent_mfma_supported(int act, int dim, int vdim, int rp);        // dim: with the rotated part
int latent_pad(int n);                                                 // padded value head size of the prefill kernel, 0 = none
int latent_key_pad(int n);                                             // of a key head (with its rotated part)
int launch_latent_decode(const LatentCall& c, hipStream_t st);         // one-token segments
int launch_latent_gather(const LatentCall& c, void* dst, hipStream_t st);   // cached + new latents of the chunks, contiguous
int launch_latent_prefill(const LatentCall& c, hipStream_t st);        // segments of two tokens and more
constexpr int LATENT_GT = 64;    // keys per gather tile

// Grouped-query attention (gqa.hip): q and k divided by their root mean square and rotated (or in the other order), scores
//   softcap tanh(q.k scale / softcap) - slope_h (i - j),  j <= i in i's own chunk of positions, or in i's window, or kept,
// exp(sink_h) in the denominator, values mixed with an earlier layer's of the same token, the output times sigmoid(gate), element by
// element or one number per head.  Every mechanism can be off.
// K and V arenas of the layer: [place][G][..][kdp] / [vdp] as AttnShape sk / sv address them.
struct GqaCall {
  SegTables t;
  AttnShape sk, sv;              // cache addressing of the keys (D = kdp) and of the values (D = vdp)
  int H, G, dim, vdim, kdp, vdp;
  const void* proj; int ldp;     // [R][ldp] outputs of the fused input projection
  int o_q, o_k, o_v, o_g;        // o_g < 0: no gate
  int gate_head;                 // 1: one gate per head
  int shared;                    // 1: keys and values are another layer's, whose cache holds this call's tokens already
  const float* q_norm; const float* k_norm; float eps;
  int rot, pairs; const float2* rot_tab;   // rotated coordinates (0: none), MI_ROT_*, [position][rot / 2] cosine and sine
  float rot_gain2;               // weight of a rotated coordinate in the mean square: 1, or (norm behind the rotation) the table's gain squared
  float scale, softcap;          // softcap 0: none
  const float* slopes;           // [H]
  const float* sink;             // [H], or null
  int chunk;                     // 0: causal only
  int window, keep;              // window 0: no window (keep is 0 then, and chunk is 0 where window is not)
  const float* v_mix;            // weight of v_first, or null
  const void* v_first_in;        // [R][G vdim] values of the first mixing layer (v_mix non-null)
  void* v_first_out;             // this layer IS the first mixing layer: its values go here; or null
  void* kcache; void* vcache;
  void* q;                       // [R][H][kdp] normed queries (prefill, generic form)
  int all_tokens;                // gqa_pre: also the one-token segments (generic form)
  float* partial; int* counters; int nsplit;      // decode: [nd][H][nsplit][vdp + 2], [nd][G head tiles] zero between launches
  void* cat; int ldc;
  int act;
};
int gqa_pad(int n);                                         // padded head size in the cache
bool gqa_mfma_supported(int act, int dim, int vdim);
bool gqa_supported(int dim, int vdim);
int launch_gqa_pre(const GqaCall& c, hipStream_t st);       // norms, value mix, append to the cache
int launch_gqa_generic(const GqaCall& c, hipStream_t st);   // any size and dtype, all tokens (after gqa_pre)
int launch_gqa_prefill(const GqaCall& c, hipStream_t st);   // segments of two tokens and more (after gqa_pre)
int launch_gqa_decode(const GqaCall& c, hipStream_t st);    // one-token segments, norms and append included
inline int gqa_head_tiles(int H, int G) { return (H / G + 15) / 16; }

// Norm of a sublayer's output + residual update + operand of what follows (layer_rows.hip):
//   x += norm(y) ;  h = next.w ? norm'(x) : x            kind: MI_NORM_*
// y comes from `y` or is the weighted sum of the experts' outputs; `router` non-null: the routing of the row as well (by x, or by h as
// stored where next.w is set).
struct PostNormW { const float* w; const float* b; int stride; };     // b: layer norm only
struct RouteArgs { int experts, top, groups, keep; const float* bias; };      // bias [experts] or null
struct PostNormCall {
  int rows;
  const float* y;                // [rows][ld], or null: parts
  const void* parts;             // [rows * top (+ rows)][ld]: routed outputs of row r at r * top + j, shared ones behind them
  const float* part_w;           // [rows][top]
  int top, shared;
  int kind; float eps;
  PostNormW norm, next;
  int width, ld;
  float* x; void* h;
  int32_t* clear; int n_clear;   // words set to zero, or null
  RouteArgs r; const void* router; int32_t* ids; float* wts;          // router [experts][ld] in the activation dtype
  int act;
};
int launch_post_norm(const PostNormCall& c, hipStream_t st);
// logits = softcap(scale * logits) in place
int launch_logit_cap(float* logits, size_t n, float scale, float softcap, hipStream_t st);

// Mixture of experts (moe.hip).  A slot is one (token, expert) pair: r * top + j for the routed ones, R * top + r for the shared.
constexpr int MOE_MAX_EXPERTS = 512, MOE_MAX_TOP = 64;
constexpr int MOE_STREAM_ROWS = 64;      // calls of up to so many tokens stream the weights, longer ones go through the tile GEMM
struct MoeCall {
  int R, width, ld;              // ld: padded width
  RouteArgs r;
  const float* x;                // [R][ld] residual stream (router), or null: the router reads h
  const void* h;                 // [R][ld] the same in the activation dtype
  const void* router;            // [experts][ld]
  int32_t* ids; float* wts;      // [R][top]
  LinearW gu, dn;                // routed: [experts][gate ffp | up ffp][ld], [experts][ld][ffp]
  LinearW sgu, sdn;              // shared: [gate sffp | up sffp][ld], [ld][sffp] (sffp = 0: none)
  int ffp, sffp, lda;            // lda: row stride of `mid`
  void* mid;                     // [slots][lda] activations
  void* out;                     // [slots][ld]
  int32_t* plan;                 // moe_plan_ints() words: tile table, sorted slots, their tokens
  int32_t* counts;               // [experts] slots per expert, [R][top] a slot's place among its expert's: left by launch_route, whose
                                 // caller clears the counts first (launch_post_norm: `clear`)
  int act;
  Glu glu;                       // the experts' unit
};
size_t moe_plan_ints(int R, const RouteArgs& r, int shared);
inline size_t moe_count_ints(int R, const RouteArgs& r) { return (size_t)r.experts + (size_t)R * r.top; }
bool moe_mfma_supported(const MoeCall& c);
int launch_route(const MoeCall& c, hipStream_t st);         // many rows of 16-bit models (few: launch_post_norm)
bool route_fused(int act, int rows, int experts);           // launch_post_norm does the routing
int launch_moe_plan(const MoeCall& c, hipStream_t st);      // many rows: order of the slots (nothing otherwise)
int launch_moe_up(const MoeCall& c, hipStream_t st);        // mid[slot] = glu(W_gate h, W_up h)
int launch_moe_down(const MoeCall& c, hipStream_t st);      // out[slot] = W_down mid[slot]

// Linear attention with a fixed decay per head (lightning.hip): S <- decay S + k v^T, o = S^T q, out = rms(o of all heads) * norm *
// sigmoid(gate).  q, k and v have been through silu.  The state is kept transposed: [value column][key channel].
constexpr int LIGHT_QT = 64;     // queries per tile; a chunk is a multiple of it
struct LightCall {
  SegTables t;
  int H, d, e;
  const void* proj; int ldp, o_q, o_k, o_v, o_g;
  const float* decay;            // [H]
  const float* log2_decay;       // [H], -1e4 for a decay of zero
  const float* norm; float eps;  // [H e]
  float* state; int sd;          // [cache row][H][e][sd], sd = d rounded up to 4
  float* o; int ldo;             // [R][ldo] outputs of the heads
  int* tickets;                  // [nd] zero between launches
  float* ws;                     // [chunks][H][padded e][padded d]: what a chunk adds to the state, then the state in front of it; null: token by token
  const int32_t* ctile; const int32_t* cbase; int nct, chunk;      // chunks of the longer segments: segment, first token; [n] a segment's first; their length
  void* cat; int ldc;
  int act;
};
bool light_supported(int d, int e);
size_t light_ws_floats(int act, int H, int d, int e);       // per chunk, 0 = token by token only
int launch_lightning(const LightCall& c, hipStream_t st);

// dst[b * db + i * di + j * dj] = src[b * sb + i * si + j * sj] for an [nb][ni][nj] box of es-byte elements
struct PlaceCall { const void* src; void* dst; int nb, ni, nj, es; size_t sb, si, sj, db, di, dj; };
int launch_place(const PlaceCall& c, hipStream_t st);

}  // namespace mi
