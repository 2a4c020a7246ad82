// engine_layers.hip -- layer-list models (MI_ARCH_LAYERS): a stack whose layers differ in mixer and sizes.
//
// What a layer launches, in order -- parallel block, x += mixer(norm(x)) + ff(norm(x)):
//   in        every projection of the normed input as ONE matrix (q | k | v | gates | feed-forward up)
//   mixer     delta.hip or latent.hip; the feed-forward activation rides in one of its launches
//   out       [mixer output | activation] times [W_o | W_down] side by side: ONE matrix, added to the float32 residual stream
//   rows      per-layer token input, residual update and the norm in front of the next layer (layer_rows.hip)
// post-norm block, x += norm1(mixer(x)), x += norm2(ff(x)):
//   in        every projection of x as ONE matrix (q | k | v | gate)
//   mixer     gqa.hip, delta.hip or latent.hip
//   out       W_o, float32
//   rows      norm1, residual update, router of the experts (layer_rows.hip; many rows: the router in moe.hip)
//   experts   gate | up of all routed experts and the shared one in one launch, down in another (moe.hip)
//   rows      weighted sum over the experts, norm2, residual update
// pre-norm block, x += m mixer(norm1(x)), x += m ff(norm2(x)), or with several streams (hyper-connections):
//   in        every projection of the normed input as ONE matrix (q | k | v | ..); the outer maps of a low-rank decay and gate as another
//   mixer     gqa.hip, delta.hip or latent.hip
//   out       W_o, float32
//   rows      update of all streams, the next sublayer's input from them, its norm (layer_rows.hip)
//   gate_up   gate | up with the activation in the epilogue;  down, float32
//   rows      as above
// sandwich block, x += norm1b(mixer(norm1(x))), x += norm2b(ff(norm2(x))): the launches of a post-norm block, whose row kernel also makes
// the norm in front of what follows; latent queries add `uq`; the feed-forward is the experts of a post-norm block or the two
// matrices of a pre-norm one
// A layer may run several times in a row; every run has a cache or state of its own (LayerRun).
// The matrices go through gemv_rows like every other linear of the engine.  A call is a list of segments (tokens of one
// cache row each), so prefill, decode and mixed steps are the same pass.
#include <cmath>

#include "engine.h"
#include "layer_kernels.h"

namespace mi {

namespace {

int up(int n, int m) { return (n + m - 1) / m * m; }

int part(PackedLinear& L, const std::string& name, int row0, int col0, int rows, int cols) {
  L.parts.push_back(PackedPart{name, row0, col0, rows, cols, false});
  return row0;
}
// a part below the ones that are there (rows padded so that every part starts at a multiple of 16)
int part_below(PackedLinear& L, const std::string& name, int rows, int pad = 16) {
  const int at = L.N;
  part(L, name, at, 0, rows, -1);
  L.N += up(rows, pad);
  return at;
}

void free_packed(PackedLinear& L) { free_linear(L.f); }

size_t act_size(const mi_engine* e) { return dtype_size(e->d.act_dtype); }

int check_matrix(const std::string& name, const int64_t* shape, int ndim, int rows, int cols) {
  if (ndim != 2 || shape[0] != rows || shape[1] != cols)
    return fail(MI_ERR_INVALID, name + ": expected shape [" + std::to_string(rows) + ", " + std::to_string(cols) + "]");
  return MI_OK;
}

int ensure_packed(mi_engine* e, PackedLinear& L) {
  if (L.f.w != nullptr) return MI_OK;
  const size_t bytes = (size_t)L.N * L.K * act_size(e);
  MI_HIP(hipMalloc(&L.f.w, bytes));
  MI_HIP(hipMemsetAsync(L.f.w, 0, bytes, e->stream));
  L.f.n_parts = 1; L.f.part_rows[0] = L.N; L.f.quant = false; L.f.dense_dtype = e->d.act_dtype; L.f.w_bytes = bytes;
  return MI_OK;
}

int put_rect(mi_engine* e, PackedLinear& L, int row0, int col0, int rows, int cols, const void* src, int on_device) {
  MI_TRY(ensure_packed(e, L));
  const size_t es = act_size(e);
  MI_HIP(hipMemcpy2DAsync((char*)L.f.w + ((size_t)row0 * L.K + col0) * es, (size_t)L.K * es, src, (size_t)cols * es, (size_t)cols * es,
                          rows, on_device ? hipMemcpyDeviceToDevice : hipMemcpyHostToDevice, e->stream));
  MI_HIP(hipStreamSynchronize(e->stream));
  return MI_OK;
}

// raw row-major copy of a matrix, optionally with a padded row stride (padding zero)
int put_raw(mi_engine* e, void*& dst, int rows, int cols, int ld, const void* src, int on_device) {
  const size_t es = act_size(e);
  if (dst == nullptr) {
    MI_HIP(hipMalloc(&dst, std::max<size_t>(16, (size_t)rows * ld * es)));
    MI_HIP(hipMemsetAsync(dst, 0, (size_t)rows * ld * es, e->stream));
  }
  MI_HIP(hipMemcpy2DAsync(dst, (size_t)ld * es, src, (size_t)cols * es, (size_t)cols * es, rows,
                          on_device ? hipMemcpyDeviceToDevice : hipMemcpyHostToDevice, e->stream));
  MI_HIP(hipStreamSynchronize(e->stream));
  return MI_OK;
}

// device copy of a host / device tensor (the caller frees it)
int stage(mi_engine* e, const void* src, size_t bytes, int on_device, void** out) {
  MI_HIP(hipMalloc(out, std::max<size_t>(16, bytes)));
  const int rc = copy_in(*out, src, bytes, on_device, e->stream);
  if (rc != MI_OK) { hipFree(*out); *out = nullptr; }
  return rc;
}

int set_vec(mi_engine* e, Vec32& v, const std::string& name, const void* data, const int64_t* shape, int ndim, int dtype, int on_device) {
  int64_t n = 1;
  for (int i = 0; i < ndim; ++i) n *= shape[i];
  if (n != v.n) return fail(MI_ERR_INVALID, name + ": expected " + std::to_string(v.n) + " elements");
  if (dtype != MI_F32 && dtype != MI_BF16 && dtype != MI_F16) return fail(MI_ERR_INVALID, name + ": bad dtype");
  if (v.p == nullptr) MI_HIP(hipMalloc(&v.p, (size_t)n * sizeof(float)));
  if (dtype == MI_F32) { MI_TRY(copy_in(v.p, data, (size_t)n * 4, on_device, e->stream)); }
  else {
    void* tmp = nullptr;
    MI_TRY(stage(e, data, (size_t)n * dtype_size(dtype), on_device, &tmp));
    const int rc = launch_convert(tmp, dtype, v.p, MI_F32, (size_t)n, e->stream);
    hipStreamSynchronize(e->stream);
    hipFree(tmp);
    MI_TRY(rc);
  }
  if (v.add != 0.f) {
    std::vector<float> host((size_t)n);
    MI_HIP(hipMemcpyAsync(host.data(), v.p, (size_t)n * 4, hipMemcpyDeviceToHost, e->stream));
    MI_HIP(hipStreamSynchronize(e->stream));
    for (float& x : host) x += v.add;
    MI_TRY(copy_in(v.p, host.data(), (size_t)n * 4, 0, e->stream));
    MI_HIP(hipStreamSynchronize(e->stream));
  }
  v.seen = true;
  return MI_OK;
}

// src [rows][cols] -> dst through launch_place (a permuted / padded copy in device memory)
int put_placed(mi_engine* e, void*& dst, size_t dst_elems, const void* src, size_t src_elems, int on_device, PlaceCall pc) {
  const size_t es = act_size(e);
  if (dst == nullptr) {
    MI_HIP(hipMalloc(&dst, std::max<size_t>(16, dst_elems * es)));
    MI_HIP(hipMemsetAsync(dst, 0, dst_elems * es, e->stream));
  }
  void* tmp = nullptr;
  MI_TRY(stage(e, src, src_elems * es, on_device, &tmp));
  pc.src = tmp; pc.dst = dst; pc.es = (int)es;
  const int rc = launch_place(pc, e->stream);
  hipStreamSynchronize(e->stream);
  hipFree(tmp);
  return rc;
}

void name_vec(Vec32& v, const std::string& name, int n) { v.name = name; v.n = n; }

// the table of cosines and sines of a layer's rotation, one per set of constants; its gain
int rotation_table(mi_engine* e, ListLayer& l) {
  const mi_layer_desc& m = l.d;
  mi_engine::RotTab key{m.rot_dims, m.rot_base, 0.f, 0.f, 0.f, 0.f, 1.f, nullptr};
  if (m.rot_factor > 0.f) { key.factor = m.rot_factor; key.original = m.rot_original; key.fast = m.rot_fast; key.slow = m.rot_slow; }
  for (const auto& t : e->rot_tabs)
    if (t.dims == key.dims && t.base == key.base && t.factor == key.factor && t.original == key.original && t.fast == key.fast && t.slow == key.slow) {
      l.rot_tab = t.p; l.rot_gain = t.gain;
      return MI_OK;
    }
  const int n = m.rot_dims / 2;
  std::vector<double> freq(n);
  for (int i = 0; i < n; ++i) freq[i] = std::pow((double)m.rot_base, -2.0 * i / m.rot_dims);
  double gain = 1.0;
  if (key.factor > 0.f) {
    // pair number (a real one) that turns `turns` times within the original context
    auto pair_of = [&](double turns) { return m.rot_dims * std::log((double)key.original / (2.0 * M_PI * turns)) / (2.0 * std::log((double)m.rot_base)); };
    const double lo = std::max(std::floor(pair_of(key.fast)), 0.0), hi = std::min(std::ceil(pair_of(key.slow)), m.rot_dims - 1.0);
    for (int i = 0; i < n; ++i) {
      const double ramp = std::min(std::max((i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
      freq[i] = freq[i] / key.factor * ramp + freq[i] * (1.0 - ramp);
    }
    gain = 0.1 * std::log((double)key.factor) + 1.0;
  }
  key.gain = (float)gain;
  MI_HIP(hipMalloc(&key.p, (size_t)e->d.max_positions * n * sizeof(float2)));
  e->rot_tabs.push_back(key);
  double* d_freq = nullptr;
  MI_HIP(hipMalloc(&d_freq, n * sizeof(double)));
  int rc = copy_in(d_freq, freq.data(), n * sizeof(double), 0, e->stream);
  if (rc == MI_OK) rc = launch_rotation_table(key.p, e->d.max_positions, n, d_freq, gain, e->stream);
  hipStreamSynchronize(e->stream);
  hipFree(d_freq);
  l.rot_tab = key.p; l.rot_gain = key.gain;
  return rc;
}

// a vector of ones that no tensor of the checkpoint sets
int set_ones(mi_engine* e, Vec32& v, int n) {
  const std::vector<float> one(n, 1.f);
  v.n = n; v.seen = true;
  MI_HIP(hipMalloc(&v.p, n * sizeof(float)));
  MI_TRY(copy_in(v.p, one.data(), n * sizeof(float), 0, e->stream));
  MI_HIP(hipStreamSynchronize(e->stream));
  return MI_OK;
}

int upload_floats(mi_engine* e, float** dst, const std::vector<float>& v) {
  MI_HIP(hipMalloc(dst, v.size() * sizeof(float)));
  MI_TRY(copy_in(*dst, v.data(), v.size() * sizeof(float), 0, e->stream));
  MI_HIP(hipStreamSynchronize(e->stream));
  return MI_OK;
}

// the unit of a feed-forward's two branches
Glu glu_of(const mi_layer_desc& m) {
  Glu g;
  if (m.act == MI_ACT_GEGLU) {
    const double c = 2.0 * std::sqrt(2.0 / M_PI);
    g.kind = GLU_GELU; g.a = (float)c; g.b = (float)(c * 0.044715);
  } else if (m.act == MI_ACT_CLAMPED) { g.kind = GLU_CLAMP; g.a = 1.702f; g.lim = m.act_limit; g.add = 1.f; }
  return g;
}

int init_layers(mi_engine* e, const mi_layer_desc* layers) {
  const mi_model_desc& d = e->d;
  e->layered = true;
  e->wp = up(d.hidden_size, 64);
  e->list.resize(d.num_layers);
  const bool mfma16 = d.act_dtype != MI_F32, post = d.block_form == MI_BLOCK_POST_NORM, pre = d.block_form == MI_BLOCK_PRE_NORM,
             both = d.block_form == MI_BLOCK_SANDWICH, serial = post || pre || both;
  const bool looped = d.loop_stop > 0;
  e->streams = std::max(1, d.streams);
  const int n_norm = d.norm_kind == MI_NORM_SCALAR ? 1 : d.hidden_size;
  int first_mix = -1;            // first layer whose values are mixed into the later ones
  for (int i = 0; i < d.num_layers; ++i) {
    ListLayer& l = e->list[i];
    l.d = layers[i];
    const mi_layer_desc& m = l.d;
    const std::string p = "l" + std::to_string(i) + ".", bad = "layer " + std::to_string(i) + ": ";
    if (m.struct_size != sizeof(mi_layer_desc)) return fail(MI_ERR_INVALID, "mi_layer_desc.struct_size does not match this library");
    if (m.heads < 1 || m.dim < 1 || m.vdim < 1 || m.ff < 0) return fail(MI_ERR_INVALID, bad + "sizes must be positive");
    const bool moe = m.ff > 0 && m.ff_kind == MI_FF_MOE;
    if (m.ff > 0 && (serial ? m.act != MI_ACT_SWIGLU && m.act != MI_ACT_GEGLU && m.act != MI_ACT_CLAMPED : m.act != MI_ACT_POLYNORM))
      return fail(MI_ERR_UNSUPPORTED, bad + "activation not supported in this block form");
    if (m.ff > 0 && m.ff_kind != (moe ? MI_FF_MOE : MI_FF_DENSE)) return fail(MI_ERR_UNSUPPORTED, bad + "unknown feed-forward kind");
    if (m.ff > 0 && !both && moe != post) return fail(MI_ERR_UNSUPPORTED, bad + "feed-forward kind not supported in this block form");
    if (m.ff > 0 && m.act == MI_ACT_CLAMPED && !(m.act_limit > 0.f)) return fail(MI_ERR_INVALID, bad + "act_limit must be positive");
    l.glu = glu_of(m);
    if (m.mixer == MI_MIXER_GQA || m.mixer == MI_MIXER_LATENT) {
      if (m.rot_dims < 0 || m.rot_dims % 2 != 0 || (m.mixer == MI_MIXER_GQA && m.rot_dims > m.dim) || (m.rot_dims > 0 && !(m.rot_base > 0.f)))
        return fail(MI_ERR_INVALID, bad + "rot_dims must be even and at most the head size, rot_base positive");
      if (m.rot_pairs != MI_ROT_HALVES && m.rot_pairs != MI_ROT_PAIRS) return fail(MI_ERR_UNSUPPORTED, bad + "unknown partners of a rotation");
      if (m.rot_factor < 0.f || (m.rot_factor > 0.f && !(m.rot_original > 0.f && m.rot_fast > 0.f && m.rot_slow > 0.f && m.rot_base != 1.f)))
        return fail(MI_ERR_INVALID, bad + "a stretched rotation needs rot_original, rot_fast and rot_slow, and a base that is not one");
      if (m.rot_dims > 0) MI_TRY(rotation_table(e, l));
    }
    l.in.K = e->wp;
    if (m.mixer == MI_MIXER_DELTA) {
      if (m.kv_heads < 1 || m.heads % m.kv_heads != 0) return fail(MI_ERR_INVALID, bad + "heads must be a multiple of kv_heads");
      if (m.conv < 1) return fail(MI_ERR_INVALID, bad + "the convolutions need at least one tap");
      if (!delta_supported(m.dim, m.vdim)) return fail(MI_ERR_UNSUPPORTED, bad + "delta rule: head sizes not supported");
      const int qk = m.kv_heads * m.dim, vv = m.heads * m.vdim;
      l.o_q = part_below(l.in, p + "mix.q", qk);
      l.o_k = part_below(l.in, p + "mix.k", qk);
      if (m.out_gate != MI_GATE_SILU && m.out_gate != MI_GATE_SIGMOID) return fail(MI_ERR_UNSUPPORTED, bad + "delta rule: unknown output gate");
      if (m.decay_rank < 0 || m.gate_rank < 0) return fail(MI_ERR_INVALID, bad + "ranks must not be negative");
      l.o_v = part_below(l.in, p + "mix.v", vv);
      if (m.gate_rank == 0) l.o_g = part_below(l.in, p + "mix.g", vv);
      l.o_b = part_below(l.in, p + "mix.b", m.heads);
      if (m.decay_rank == 0) l.o_a = part_below(l.in, p + "mix.a", m.heads);
      // inner projections padded to the tile GEMM's step, directly behind each other: the columns of the outer matrix
      auto low_rank = [&](const char* name, int rank, int rows, int& out_at) {
        if (rank == 0) return;
        const int at = part_below(l.in, p + "mix." + name + "1", rank, 64);
        if (l.o_lr < 0) l.o_lr = at;
        l.o_lrg = at;
        out_at = part(l.lr, p + "mix." + name + "2", l.lr.N, at - l.o_lr, rows, rank);
        l.lr.N += up(rows, 16);
        l.lr.K = at - l.o_lr + up(rank, 64);
      };
      low_rank("a", m.decay_rank, m.heads * m.dim, l.o_a);
      low_rank("g", m.gate_rank, vv, l.o_g);
      name_vec(l.conv_q, p + "mix.q.conv", qk * m.conv);
      name_vec(l.conv_k, p + "mix.k.conv", qk * m.conv);
      name_vec(l.conv_v, p + "mix.v.conv", vv * m.conv);
      name_vec(l.A_log, p + "mix.A_log", m.heads);
      name_vec(l.dt_bias, p + "mix.dt_bias", m.decay_rank > 0 ? m.heads * m.dim : m.heads);
      name_vec(l.head_norm, p + "mix.norm", m.vdim);
    } else if (m.mixer == MI_MIXER_LATENT) {
      if (m.kv_rank < 1 || m.kv_rank > 1024) return fail(MI_ERR_UNSUPPORTED, bad + "kv_rank must be in [1, 1024]");
      e->any_latent = true;
      l.src = i;
      if (m.kv_from >= 0) {
        if (m.kv_from >= i || layers[m.kv_from].mixer != MI_MIXER_LATENT || layers[m.kv_from].kv_from >= 0 ||
            layers[m.kv_from].kv_rank != m.kv_rank || layers[m.kv_from].rot_dims != m.rot_dims)
          return fail(MI_ERR_INVALID, bad + "kv_from must name an earlier latent-attention layer with latents of its own and the same sizes");
        if (looped) return fail(MI_ERR_UNSUPPORTED, bad + "no latents of another layer in a looped stack");
        l.src = m.kv_from;
      }
      const int qd = m.dim + m.rot_dims;
      l.cp = up(m.kv_rank, 16);
      l.rp = up(l.cp + m.rot_dims, 64);
      if (l.rp > 1024) return fail(MI_ERR_UNSUPPORTED, bad + "latent and rotated part above 1024");
      if (m.q_rank < 0) return fail(MI_ERR_INVALID, bad + "q_rank must not be negative");
      if (m.out_gate != MI_GATE_NONE && m.out_gate != MI_GATE_SIGMOID_HEAD) return fail(MI_ERR_UNSUPPORTED, bad + "latent attention: unknown output gate");
      if (m.q_rank > 0) {
        l.o_qc = part_below(l.in, p + "mix.dq", m.q_rank);
        l.qr = up(m.q_rank, 64);
        name_vec(l.dq_norm, p + "mix.dq.norm", m.q_rank);
        part(l.uq, p + "mix.uq", 0, 0, m.heads * qd, m.q_rank);
        l.uq.N = up(m.heads * qd, 16); l.uq.K = l.qr;
      } else l.o_q = part_below(l.in, p + "mix.q", m.heads * qd);
      if (m.out_gate != MI_GATE_NONE) l.o_g = part_below(l.in, p + "mix.g", m.heads);
      if (m.kv_from < 0) {
        l.o_c = part_below(l.in, p + "mix.dkv", m.kv_rank + m.rot_dims);
        name_vec(l.c_norm, p + "mix.dkv.norm", m.kv_rank);
      }
      if (mfma16 && m.scale > 0.f && latent_mfma_supported(d.act_dtype, qd, m.vdim, l.rp)) {
        l.kdp = latent_key_pad(qd); l.vdp = latent_pad(m.vdim);
        e->latent_qt = std::min(e->latent_qt, latent_tile(l.kdp, l.vdp));
        l.ukv.K = l.rp; l.ukv.N = m.heads * (l.kdp + l.vdp);
      }
    } else if (m.mixer == MI_MIXER_GQA) {
      if (!serial) return fail(MI_ERR_UNSUPPORTED, bad + "grouped-query attention is no mixer of parallel blocks");
      if (m.kv_heads < 1 || m.heads % m.kv_heads != 0) return fail(MI_ERR_INVALID, bad + "heads must be a multiple of kv_heads");
      if (!gqa_supported(m.dim, m.vdim)) return fail(MI_ERR_UNSUPPORTED, bad + "grouped-query attention: head sizes not supported");
      if (m.chunk < 0 || m.softcap < 0.f || m.window < 0 || m.keep_first < 0) return fail(MI_ERR_INVALID, bad + "chunk, window, keep_first and softcap must not be negative");
      if (m.chunk > 0 && m.window > 0) return fail(MI_ERR_UNSUPPORTED, bad + "chunks and a sliding window in one layer");
      if (m.out_gate != MI_GATE_NONE && m.out_gate != MI_GATE_SIGMOID && m.out_gate != MI_GATE_SIGMOID_HEAD) return fail(MI_ERR_UNSUPPORTED, bad + "grouped-query attention: unknown output gate");
      if (looped && m.v_mix) return fail(MI_ERR_UNSUPPORTED, bad + "no mixed values in a looped stack");
      if (m.qk_norm != MI_QK_NORM_FIRST && m.qk_norm != MI_QK_NORM_LAST) return fail(MI_ERR_UNSUPPORTED, bad + "unknown norm of queries and keys");
      l.src = i;
      if (m.kv_from >= 0) {
        if (m.kv_from >= i || layers[m.kv_from].mixer != MI_MIXER_GQA || layers[m.kv_from].kv_from >= 0 || layers[m.kv_from].kv_heads != m.kv_heads ||
            layers[m.kv_from].dim != m.dim || layers[m.kv_from].vdim != m.vdim)
          return fail(MI_ERR_INVALID, bad + "kv_from must name an earlier grouped-query layer with keys and values of its own and the same sizes");
        if (looped || m.v_mix) return fail(MI_ERR_UNSUPPORTED, bad + "no keys and values of another layer in a looped stack or with mixed values");
        l.src = m.kv_from;
      }
      l.kdp = gqa_pad(m.dim); l.vdp = gqa_pad(m.vdim);
      l.gqa_fast = gqa_mfma_supported(d.act_dtype, m.dim, m.vdim);
      l.o_q = part_below(l.in, p + "mix.q", m.heads * m.dim);
      if (m.kv_from < 0) {
        l.o_k = part_below(l.in, p + "mix.k", m.kv_heads * m.dim);
        l.o_v = part_below(l.in, p + "mix.v", m.kv_heads * m.vdim);
      }
      if (m.out_gate != MI_GATE_NONE) l.o_g = part_below(l.in, p + "mix.g", m.out_gate == MI_GATE_SIGMOID_HEAD ? m.heads : m.heads * m.vdim);
      if (m.sink) name_vec(l.sink, p + "mix.sink", m.heads);
      if (m.qk_norm == MI_QK_NORM_FIRST) {
        name_vec(l.q_norm, p + "mix.q.norm", m.dim);
        name_vec(l.k_norm, p + "mix.k.norm", m.dim);
      } else {
        MI_TRY(set_ones(e, l.q_norm, m.dim));
        MI_TRY(set_ones(e, l.k_norm, m.dim));
      }
      if (m.v_mix) {
        name_vec(l.vmix, p + "mix.vmix", 1);
        if (first_mix < 0) { first_mix = i; l.v_first = true; l.vmix.optional = true; }
        else if (layers[first_mix].kv_heads * layers[first_mix].vdim != m.kv_heads * m.vdim)
          return fail(MI_ERR_INVALID, bad + "mixed values must have the size of the first such layer's");
        e->n_vfirst = m.kv_heads * m.vdim;
      }
      std::vector<float> slopes(m.heads, 0.f);
      if (m.slope_exp > 0.f) for (int h = 0; h < m.heads; ++h) slopes[h] = (float)std::pow(2.0, -(double)m.slope_exp * (h + 1) / m.heads);
      MI_TRY(upload_floats(e, &l.slopes, slopes));
      if (e->gqa_chunk < 0) { e->gqa_chunk = m.chunk; e->gqa_window = m.window; }
    } else if (m.mixer == MI_MIXER_LIGHTNING) {
      if (!serial) return fail(MI_ERR_UNSUPPORTED, bad + "lightning attention is no mixer of parallel blocks");
      if (!light_supported(m.dim, m.vdim)) return fail(MI_ERR_UNSUPPORTED, bad + "lightning attention: head sizes not supported");
      if (m.out_gate != MI_GATE_SIGMOID) return fail(MI_ERR_UNSUPPORTED, bad + "lightning attention: unknown output gate");
      if (m.decay == nullptr) return fail(MI_ERR_INVALID, bad + "lightning attention needs a decay per head");
      std::vector<float> dec(m.heads), lg(m.heads);
      for (int h = 0; h < m.heads; ++h) {
        if (!(m.decay[h] >= 0.0 && m.decay[h] <= 1.0)) return fail(MI_ERR_INVALID, bad + "a decay must be in [0, 1]");
        dec[h] = (float)m.decay[h];
        lg[h] = (float)std::max(-1e4, std::log2(m.decay[h]));
      }
      l.d.decay = nullptr;                           // (the caller's)
      MI_TRY(upload_floats(e, &l.decay, dec));
      MI_TRY(upload_floats(e, &l.log2_decay, lg));
      l.sd = up(m.dim, 4);
      l.o_q = part_below(l.in, p + "mix.q", m.heads * m.dim);
      l.o_k = part_below(l.in, p + "mix.k", m.heads * m.dim);
      l.o_v = part_below(l.in, p + "mix.v", m.heads * m.vdim);
      l.o_g = part_below(l.in, p + "mix.g", m.heads * m.vdim);
      name_vec(l.head_norm, p + "mix.norm", m.heads * m.vdim);
      e->any_light = true;
    } else return fail(MI_ERR_UNSUPPORTED, bad + "unknown mixer");
    const int hv = m.heads * m.vdim;
    part(l.out, p + "mix.o", 0, 0, d.hidden_size, hv);
    l.n_cat = up(hv, 64);
    if (moe) {
      if (m.experts < 1 || m.experts > MOE_MAX_EXPERTS || m.top < 1 || m.top > MOE_MAX_TOP || m.groups < 1 || m.experts % m.groups != 0 ||
          m.keep < 1 || m.keep > m.groups || m.top > m.keep * (m.experts / m.groups) || m.shared_ff < 0)
        return fail(MI_ERR_INVALID, bad + "experts, top, groups and keep do not fit each other (at most 512 experts, 64 of them per token)");
      if (m.router_bias) name_vec(l.router_b, p + "mlp.router.b", m.experts);
      l.ffp = up(m.ff, 64); l.sffp = up(m.shared_ff, 64);
      l.gu.K = l.sgu.K = e->wp;
      l.dn.K = l.ffp; l.sdn.K = l.sffp;
      for (int x = 0; x < m.experts; ++x) {
        const std::string pe = p + "mlp.e" + std::to_string(x) + ".";
        part(l.gu, pe + "gate", x * 2 * l.ffp, 0, m.ff, d.hidden_size);
        part(l.gu, pe + "up", x * 2 * l.ffp + l.ffp, 0, m.ff, d.hidden_size);
        part(l.dn, pe + "down", x * e->wp, 0, d.hidden_size, m.ff);
      }
      l.gu.N = m.experts * 2 * l.ffp; l.dn.N = m.experts * e->wp;
      if (m.shared_ff > 0) {
        part(l.sgu, p + "mlp.shared.gate", 0, 0, m.shared_ff, d.hidden_size);
        part(l.sgu, p + "mlp.shared.up", l.sffp, 0, m.shared_ff, d.hidden_size);
        part(l.sdn, p + "mlp.shared.down", 0, 0, d.hidden_size, m.shared_ff);
        l.sgu.N = 2 * l.sffp; l.sdn.N = e->wp;
      }
    } else if (m.ff > 0 && serial) {
      l.ffp = up(m.ff, 64);
      part(l.gu, p + "mlp.gate", 0, 0, m.ff, d.hidden_size);
      part(l.gu, p + "mlp.up", l.ffp, 0, m.ff, d.hidden_size);
      part(l.dn, p + "mlp.down", 0, 0, d.hidden_size, m.ff);
      l.gu.N = 2 * l.ffp; l.gu.K = e->wp;
      l.dn.N = e->wp; l.dn.K = l.ffp;
    } else if (m.ff > 0) {
      l.o_up = part_below(l.in, p + "mlp.up", m.ff);
      l.o_ff = l.n_cat;
      part(l.out, p + "mlp.down", 0, l.o_ff, d.hidden_size, m.ff);
      l.n_cat += up(m.ff, 64);
      name_vec(l.act, p + "mlp.act", 4);
    }
    for (auto& q : l.in.parts) if (q.cols < 0) q.cols = d.hidden_size;
    l.out.N = e->wp; l.out.K = l.n_cat;
    name_vec(l.norm, p + "norm1", n_norm);
    if (serial && m.ff > 0) name_vec(l.norm2, p + "norm2", n_norm);
    if (both) name_vec(l.norm_out, p + "norm1b", n_norm);
    if (both && m.ff > 0) name_vec(l.norm2_out, p + "norm2b", n_norm);
    l.norm.add = l.norm2.add = l.norm_out.add = l.norm2_out.add = d.norm_offset ? 1.f : 0.f;
    for (int q = 0; q < 2 && d.streams > 0; ++q) {
      if (q == 1 && m.ff == 0) break;
      const std::string ph = p + "hc" + std::to_string(q + 1) + ".";
      name_vec(l.hc_in[q], ph + "in", d.streams);
      name_vec(l.hc_mix[q], ph + "mix", d.streams * d.streams);
      name_vec(l.hc_out[q], ph + "out", d.streams);
    }
    if (d.norm_kind == MI_NORM_LAYER) {
      name_vec(l.norm_b, p + "norm1.b", n_norm);
      if (m.ff > 0) name_vec(l.norm2_b, p + "norm2.b", n_norm);
    }
    if (d.side_dim > 0) name_vec(l.side_norm, p + "side.norm", d.hidden_size);
  }
  for (int i = 0; i < d.num_layers; ++i) {             // the order of the runs, and what each keeps
    const int stop = looped ? d.loop_stop : 0;
    if (looped && i == d.loop_start) {
      for (int pass = 0; pass < d.loop_times; ++pass)
        for (int j = d.loop_start; j < stop; ++j) e->runs.push_back(LayerRun{j});
      i = stop - 1;
    } else e->runs.push_back(LayerRun{i});
  }
  for (LayerRun& r : e->runs) {
    const mi_layer_desc& m = e->list[r.layer].d;
    if (m.mixer == MI_MIXER_DELTA || m.mixer == MI_MIXER_LIGHTNING) r.state = e->n_state++;
    else if (m.kv_from >= 0) continue;
    else if (m.mixer == MI_MIXER_GQA) { r.k = e->n_arena++; r.v = e->n_arena++; }
    else r.lat = e->n_arena++;
  }
  name_vec(e->list_final_norm, "final.norm", n_norm);
  e->list_final_norm.add = d.norm_offset ? 1.f : 0.f;
  if (d.norm_kind == MI_NORM_LAYER) name_vec(e->list_final_norm_b, "final.norm.b", n_norm);
  e->list_head.K = e->wp; e->list_head.N = d.vocab_size;
  part(e->list_head, "head", 0, 0, d.vocab_size, d.hidden_size);
  const int nf = (d.hidden_size + 1) / 2;
  std::vector<double> freq(nf);
  for (int i = 0; i < nf; ++i) freq[i] = std::pow(10000.0, -2.0 * i / d.hidden_size);
  if (d.position == MI_POS_SINUSOIDAL) {
    MI_HIP(hipMalloc(&e->d_freq, nf * sizeof(double)));
    MI_TRY(copy_in(e->d_freq, freq.data(), nf * sizeof(double), 0, e->stream));
  }
  return MI_OK;
}

template <typename F>
void each_vec(mi_engine* e, F f) {
  for (auto& l : e->list)
    for (Vec32* v : {&l.norm, &l.act, &l.conv_q, &l.conv_k, &l.conv_v, &l.A_log, &l.dt_bias, &l.head_norm, &l.c_norm, &l.side_norm,
                     &l.q_norm, &l.k_norm, &l.vmix, &l.norm_b, &l.norm2, &l.norm2_b, &l.sink, &l.hc_in[0], &l.hc_in[1], &l.hc_mix[0], &l.hc_mix[1],
                     &l.hc_out[0], &l.hc_out[1], &l.dq_norm, &l.norm_out, &l.norm2_out, &l.router_b}) f(*v);
  f(e->list_final_norm);
  f(e->list_final_norm_b);
}

int finalize_packed(mi_engine* e, PackedLinear& L) {
  for (auto& q : L.parts) if (!q.seen) return fail(MI_ERR_NOTFOUND, q.name + ": weight not set");
  L.f.seen_w[0] = 1;
  return finalize_linear(e, L.f, L.K, L.parts.empty() ? "packed" : L.parts[0].name);
}

// ---- per-call tables ------------------------------------------------------------------------------------------------
constexpr int DELTA_CHUNK_FROM = 24;     // longest portion of a call from which the delta rule goes chunk by chunk
constexpr int LIGHT_LONG = 8192;         // tokens of a call from which lightning attention takes chunks of 256 instead of 128
struct Tables {
  SegTables t;
  int nkeys = 0, maxlen = 0;
  const int32_t* full = nullptr; int nfull = 0, qfull = 0;     // query tiles without a window or chunks, and their size (latent attention)
  const int32_t* lchunk = nullptr; const int32_t* lbase = nullptr; int nl = 0, lsize = 0;      // chunks of the lightning attention
};

int build_tables(mi_engine* e, mi_kv* kv, const int32_t* rows, const int32_t* lens, int n, Tables& out) {
  SegTables& t = out.t;
  t.n = n; t.R = 0;
  std::vector<int32_t> tok0(n), kbase(n, 0), cbase(n, 0), tok_seg, dec, chunk, tile, full, gt, ct, lc, lbase(n, 0);
  int total = 0;
  for (int i = 0; i < n; ++i) total += lens[i];
  out.lsize = total >= LIGHT_LONG ? 256 : 128;
  for (int i = 0; i < n; ++i) {
    tok0[i] = t.R;
    for (int j = 0; j < lens[i]; ++j) tok_seg.push_back(i);
    t.R += lens[i];
    if (lens[i] == 1) { dec.push_back(i); continue; }
    chunk.push_back(i);
    kbase[i] = out.nkeys;
    const int keys = kv->h_off[rows[i]] + lens[i];
    out.nkeys += keys;
    for (int k = 0; k < keys; k += LATENT_GT) { gt.push_back(i); gt.push_back(k); }
    cbase[i] = (int)ct.size() / 2;
    for (int k = 0; k < lens[i]; k += DELTA_CHUNK) { ct.push_back(i); ct.push_back(k); }
    lbase[i] = (int)lc.size() / 2;
    for (int k = 0; e->any_light && k < lens[i]; k += out.lsize) { lc.push_back(i); lc.push_back(k); }
  }
  int longest = 0;
  for (int i : chunk) longest = std::max(longest, lens[i]);
  out.qfull = longest >= 256 ? e->latent_qt : 64;
  t.qt = 64;                                     // (gqa.hip has the small tile only)
  // the tiles with the most keys in front of them first (attention over chunks of positions: within the chunk, over a window: within it)
  struct Tile { int keys, seg, q; };
  auto tiles = [&](std::vector<int32_t>& dst, int qt, int cut, int window) {
    std::vector<Tile> order;
    for (int i : chunk)
      for (int q = (lens[i] - 1) / qt * qt; q >= 0; q -= qt) {
        const int p0 = kv->h_off[rows[i]] + q, p1 = kv->h_off[rows[i]] + std::min(q + qt, lens[i]);
        order.push_back(Tile{cut > 0 ? p1 - p0 / cut * cut : (window > 0 ? std::min(p1, p1 - p0 + window) : p1), i, q});
      }
    std::stable_sort(order.begin(), order.end(), [](const Tile& a, const Tile& b) { return a.keys > b.keys; });
    for (const Tile& x : order) { dst.push_back(x.seg); dst.push_back(x.q); }
  };
  if (e->gqa_chunk >= 0) tiles(tile, t.qt, e->gqa_chunk, e->gqa_window);
  if (e->any_latent) tiles(full, out.qfull, 0, 0);
  std::vector<int32_t> m;
  auto add = [&](const int32_t* p, size_t k) { const size_t at = m.size(); m.insert(m.end(), p, p + k); while (m.size() % 4) m.push_back(0); return at; };
  const size_t a_row = add(rows, n), a_t0 = add(tok0.data(), n), a_len = add(lens, n), a_kb = add(kbase.data(), n), a_cb = add(cbase.data(), n),
               a_ts = add(tok_seg.data(), tok_seg.size()), a_dec = add(dec.data(), dec.size()), a_ch = add(chunk.data(), chunk.size()),
               a_ti = add(tile.data(), tile.size()), a_gt = add(gt.data(), gt.size()),
               a_ct = add(ct.data(), ct.size()), a_fu = add(full.data(), full.size()), a_lc = add(lc.data(), lc.size()),
               a_lb = add(lbase.data(), n);
  if (m.size() > e->d_meta_cap) {
    MI_HIP(hipStreamSynchronize(e->stream));
    hipFree(e->d_meta); e->d_meta = nullptr; e->d_meta_cap = 0;
    const size_t cap = std::max<size_t>(2 * m.size(), 4096);
    MI_HIP(hipMalloc(&e->d_meta, cap * sizeof(int32_t)));
    e->d_meta_cap = cap;
    e->h_meta.clear();
  }
  if (m != e->h_meta) {        // (a decode loop over an unchanged row set uploads nothing)
    MI_HIP(hipMemcpyAsync(e->d_meta, m.data(), m.size() * sizeof(int32_t), hipMemcpyHostToDevice, e->stream));
    e->h_meta = m;
  }
  const int32_t* b = e->d_meta;
  t.row = b + a_row; t.tok0 = b + a_t0; t.len = b + a_len; t.kbase = b + a_kb; t.cbase = b + a_cb; t.tok_seg = b + a_ts; t.dec = b + a_dec;
  t.chunk = b + a_ch; t.tile = b + a_ti; t.gtile = b + a_gt; t.ctile = b + a_ct; t.off = kv->d_off;
  t.nd = (int)dec.size(); t.nc = (int)chunk.size(); t.nt = (int)tile.size() / 2; t.ngt = (int)gt.size() / 2; t.nct = (int)ct.size() / 2;
  out.maxlen = longest;
  out.full = b + a_fu; out.nfull = (int)full.size() / 2;
  out.lchunk = b + a_lc; out.lbase = b + a_lb; out.nl = (int)lc.size() / 2;
  return MI_OK;
}

int grow(mi_engine* e, void** p, size_t* cap, size_t need) {
  if (need <= *cap) return MI_OK;
  MI_HIP(hipStreamSynchronize(e->stream));
  hipFree(*p); *p = nullptr; *cap = 0;
  MI_HIP(hipMalloc(p, need));
  *cap = need;
  return MI_OK;
}

int latent_nsplit(const mi_kv* kv, const int32_t* rows, const int32_t* lens, int n, int nd, int head_tiles) {
  int mx = 1;
  for (int i = 0; i < n; ++i) if (lens[i] == 1) mx = std::max(mx, kv->h_off[rows[i]] + 1);
  int ns = std::max(1, 256 / std::max(1, nd * head_tiles));
  ns = std::min(ns, (mx + 127) / 128);               // at least one 32-key block per wave of a split
  return std::max(1, std::min(ns, 32));
}

// key splits of a decode launch: enough workgroups for the chip, at least two 32-key blocks per wave
int gqa_nsplit(const mi_kv* kv, const ListLayer& l, const int32_t* rows, const int32_t* lens, int n, int nd) {
  int mx = 0;
  for (int i = 0; i < n; ++i)
    if (lens[i] == 1) {
      const int pos = kv->h_off[rows[i]];
      mx = std::max(mx, l.d.chunk > 0 ? pos % l.d.chunk : (l.d.window > 0 ? (int)std::min<int64_t>(pos, (int64_t)l.d.window + l.d.keep_first) : pos));
    }
  const int ns = std::max(1, 512 / std::max(1, nd * l.d.kv_heads * gqa_head_tiles(l.d.heads, l.d.kv_heads)));
  return std::max(1, std::min({ns, (mx + 255) / 256, 32}));
}

int run_gqa(mi_engine* e, mi_kv* kv, ListLayer& l, const LayerRun& run, const Tables& tb, const int32_t* rows, const int32_t* lens, int n) {
  const mi_model_desc& d = e->d;
  const mi_layer_desc& m = l.d;
  hipStream_t st = e->stream;
  const size_t es = dtype_size(kv->dtype);
  GqaCall c{};
  c.t = tb.t;
  c.sk = AttnShape{1, 1, m.heads, m.kv_heads, l.kdp, d.act_dtype, kv->dtype, RND_NONE, kv->cap, nullptr, nullptr, 0, 0};
  kv_shape(kv, c.sk);
  c.sv = c.sk;
  c.sv.D = l.vdp;
  c.H = m.heads; c.G = m.kv_heads; c.dim = m.dim; c.vdim = m.vdim; c.kdp = l.kdp; c.vdp = l.vdp;
  c.proj = e->proj; c.ldp = l.in.N; c.o_q = l.o_q; c.o_k = l.o_k; c.o_v = l.o_v; c.o_g = l.o_g;
  c.gate_head = m.out_gate == MI_GATE_SIGMOID_HEAD ? 1 : 0; c.shared = m.kv_from >= 0 ? 1 : 0;
  c.q_norm = l.q_norm.p; c.k_norm = l.k_norm.p; c.eps = d.rms_norm_eps;
  c.scale = m.scale; c.softcap = m.softcap; c.slopes = l.slopes; c.chunk = m.chunk;
  c.rot = m.rot_dims; c.rot_tab = l.rot_tab; c.sink = l.sink.p; c.pairs = m.rot_pairs;
  c.rot_gain2 = m.qk_norm == MI_QK_NORM_LAST ? l.rot_gain * l.rot_gain : 1.f;
  c.window = m.window; c.keep = m.window > 0 ? m.keep_first : 0;
  if (m.v_mix && l.v_first) c.v_first_out = e->v_first;
  else if (m.v_mix) { c.v_mix = l.vmix.p; c.v_first_in = e->v_first; }
  const LayerRun& src = c.shared ? e->runs[l.src] : run;         // (a layer that reads another's stands in a stack without loops: run = layer)
  c.kcache = (char*)kv->k + kv->arenas[src.k].off * es;
  c.vcache = (char*)kv->k + kv->arenas[src.v].off * es;
  c.q = e->lq; c.nsplit = 1;
  c.cat = e->cat; c.ldc = l.n_cat; c.act = d.act_dtype;
  c.all_tokens = l.gqa_fast ? 0 : 1;
  if (!l.gqa_fast || c.t.nc > 0) { Prof pr(e, "gqa_pre"); MI_TRY(launch_gqa_pre(c, st)); }
  if (!l.gqa_fast) { Prof pr(e, "gqa_generic"); return launch_gqa_generic(c, st); }
  if (c.t.nd > 0) {
    c.nsplit = gqa_nsplit(kv, l, rows, lens, n, c.t.nd);
    if (c.nsplit > 1) {
      MI_TRY(grow(e, (void**)&e->gqa_part, &e->gqa_part_cap, (size_t)c.t.nd * m.heads * c.nsplit * (l.vdp + 2) * sizeof(float)));
      const size_t ctr = (size_t)c.t.nd * m.kv_heads * gqa_head_tiles(m.heads, m.kv_heads) * sizeof(int), had = e->gqa_ctr_cap;
      MI_TRY(grow(e, (void**)&e->gqa_ctr, &e->gqa_ctr_cap, ctr));
      if (e->gqa_ctr_cap != had) MI_HIP(hipMemsetAsync(e->gqa_ctr, 0, e->gqa_ctr_cap, st));
      c.partial = e->gqa_part; c.counters = e->gqa_ctr;
    }
    Prof pr(e, "gqa_decode");
    MI_TRY(launch_gqa_decode(c, st));
  }
  if (c.t.nc > 0) { Prof pr(e, "gqa_prefill"); MI_TRY(launch_gqa_prefill(c, st)); }
  return MI_OK;
}

int run_lightning(mi_engine* e, mi_kv* kv, ListLayer& l, const LayerRun& run, const Tables& tb) {
  const mi_layer_desc& m = l.d;
  LightCall c{};
  c.t = tb.t;
  c.H = m.heads; c.d = m.dim; c.e = m.vdim;
  c.proj = e->proj; c.ldp = l.in.N; c.o_q = l.o_q; c.o_k = l.o_k; c.o_v = l.o_v; c.o_g = l.o_g;
  c.decay = l.decay; c.log2_decay = l.log2_decay; c.norm = l.head_norm.p; c.eps = e->d.rms_norm_eps;
  c.state = (float*)(kv->state + kv->state_off[run.state]); c.sd = l.sd;
  c.o = e->scan32; c.ldo = e->scan_ld;
  c.cat = e->cat; c.ldc = l.n_cat; c.act = e->d.act_dtype;
  if (c.t.nd > 0) {
    const size_t had = e->light_ctr_cap;
    MI_TRY(grow(e, (void**)&e->light_ctr, &e->light_ctr_cap, (size_t)c.t.nd * sizeof(int)));
    if (e->light_ctr_cap != had) MI_HIP(hipMemsetAsync(e->light_ctr, 0, e->light_ctr_cap, e->stream));
    c.tickets = e->light_ctr;
  }
  const size_t per = light_ws_floats(c.act, c.H, c.d, c.e);
  if (c.t.nc > 0 && per > 0) {
    MI_TRY(grow(e, (void**)&e->light_ws, &e->light_ws_cap, (size_t)tb.nl * per * sizeof(float)));
    c.ws = e->light_ws; c.ctile = tb.lchunk; c.cbase = tb.lbase; c.nct = tb.nl; c.chunk = tb.lsize;
  }
  Prof pr(e, "lightning");
  return launch_lightning(c, e->stream);
}

// the second half of a post-norm layer: experts behind the row kernel that made their input
MoeCall moe_call(mi_engine* e, const ListLayer& l, int R) {
  MoeCall c{};
  c.R = R; c.width = e->d.hidden_size; c.ld = e->wp;
  c.r = RouteArgs{l.d.experts, l.d.top, l.d.groups, l.d.keep, l.router_b.p};
  c.x = e->d.block_form == MI_BLOCK_SANDWICH ? nullptr : e->x32; c.h = e->hn; c.router = l.router; c.ids = e->moe_ids; c.wts = e->moe_wts;
  c.gu = l.gu.f.W; c.dn = l.dn.f.W; c.sgu = l.sgu.f.W; c.sdn = l.sdn.f.W;
  c.ffp = l.ffp; c.sffp = l.sffp; c.lda = std::max(l.ffp, l.sffp);
  c.mid = e->moe_mid; c.out = e->moe_out; c.plan = e->moe_plan; c.counts = e->moe_counts; c.act = e->d.act_dtype; c.glu = l.glu;
  return c;
}

int run_latent(mi_engine* e, mi_kv* kv, ListLayer& l, const Tables& tb, const int32_t* rows, const int32_t* lens, int n, LatentCall c) {
  hipStream_t st = e->stream;
  c.t.tile = tb.full; c.t.nt = tb.nfull; c.t.qt = tb.qfull;
  { Prof pr(e, "latent_pre"); MI_TRY(launch_latent_pre(c, st)); }
  if (c.q_rank > 0) {
    const size_t es = act_size(e);
    GemvCall g; g.x = c.qc; g.ldx = c.ldqc; g.act = c.act; g.epi = EPI_STORE; g.out = e->qfull; g.ldo = l.uq.N;
    MI_TRY(gemv_rows(e, l.uq.f, g, c.t.R, es, es, "latent_uq"));
  }
  if (l.kdp == 0) { Prof pr(e, "latent_generic"); return launch_latent_generic(c, st); }
  if (c.t.nd > 0) {
    const int ht = (c.H + 15) / 16;
    c.nsplit = latent_nsplit(kv, rows, lens, n, c.t.nd, ht);
    void* part_p = e->lat_part;
    MI_TRY(grow(e, &part_p, &e->lat_part_cap, (size_t)c.t.nd * ht * 16 * c.nsplit * (c.rp + 4) * sizeof(float)));
    e->lat_part = (float*)part_p;
    c.partial = e->lat_part;
    MI_TRY(grow(e, &e->lat_m, &e->lat_m_cap, (size_t)c.t.nd * c.H * 2 * c.rp * act_size(e)));
    c.merged = e->lat_m;
    Prof pr(e, "latent_decode");
    MI_TRY(launch_latent_decode(c, st));
  }
  if (c.t.nc > 0) {
    const size_t es = act_size(e);
    MI_TRY(grow(e, &e->lat_x, &e->lat_x_cap, (size_t)tb.nkeys * c.rp * es));
    MI_TRY(grow(e, &e->lat_kv, &e->lat_kv_cap, (size_t)tb.nkeys * l.ukv.N * es));
    { Prof pr(e, "latent_gather"); MI_TRY(launch_latent_gather(c, e->lat_x, st)); }
    GemvCall g; g.x = e->lat_x; g.ldx = c.rp; g.act = c.act; g.epi = EPI_STORE; g.out = e->lat_kv; g.ldo = l.ukv.N;
    const int keep = e->cur_L;
    e->cur_L = 2;
    const int rc = gemv_rows(e, l.ukv.f, g, tb.nkeys, es, es, "latent_kv");
    e->cur_L = keep;
    MI_TRY(rc);
    c.kv = e->lat_kv; c.ldkv = l.ukv.N;
    Prof pr(e, "latent_prefill");
    MI_TRY(launch_latent_prefill(c, st));
  }
  return MI_OK;
}

}  // namespace

int layers_set_tensor(mi_engine* e, const std::string& name, const void* data, const int64_t* shape, int ndim, int dtype, int on_device) {
  const mi_model_desc& d = e->d;
  // small tensors kept in float32
  Vec32* hit = nullptr;
  each_vec(e, [&](Vec32& v) { if (v.n > 0 && v.name == name) hit = &v; });
  if (hit) return set_vec(e, *hit, name, data, shape, ndim, dtype, on_device);
  // everything else is a matrix in the model dtype
  const auto dense = [&]() -> int {
    if (dtype != d.act_dtype) return fail(MI_ERR_UNSUPPORTED, name + ": weight dtype differs from the model dtype");
    return MI_OK;
  };
  auto try_packed = [&](PackedLinear& L, bool& found) -> int {
    for (auto& q : L.parts)
      if (q.name == name) {
        found = true;
        MI_TRY(dense());
        MI_TRY(check_matrix(name, shape, ndim, q.rows, q.cols));
        MI_TRY(put_rect(e, L, q.row0, q.col0, q.rows, q.cols, data, on_device));
        q.seen = true;
      }
    return MI_OK;
  };
  bool found = false;
  MI_TRY(try_packed(e->list_head, found));
  for (auto& l : e->list)
    for (PackedLinear* L : {&l.in, &l.lr, &l.uq, &l.out, &l.gu, &l.dn, &l.sgu, &l.sdn}) MI_TRY(try_packed(*L, found));
  for (int i = 0; i < d.num_layers && found; ++i) {    // (the outer low-rank maps are kept row-major as well)
    ListLayer& l = e->list[i];
    const mi_layer_desc& m = l.d;
    const std::string p = "l" + std::to_string(i) + ".mix.";
    if (!(m.mixer == MI_MIXER_DELTA && m.decay_rank > 0 && m.gate_rank > 0)) continue;
    if (name == p + "a2") MI_TRY(put_raw(e, l.low_a, m.heads * m.dim, m.decay_rank, up(m.decay_rank, 8), data, on_device));
    if (name == p + "g2") MI_TRY(put_raw(e, l.low_g, m.heads * m.vdim, m.gate_rank, up(m.gate_rank, 8), data, on_device));
  }
  if (found) return MI_OK;
  const int W = d.hidden_size;
  if (name == "embed") {
    MI_TRY(dense());
    MI_TRY(check_matrix(name, shape, ndim, d.vocab_size, W));
    MI_TRY(put_raw(e, e->tok_embed, d.vocab_size, W, W, data, on_device));
    e->tok_embed_seen = true;
    return MI_OK;
  }
  if (name == "bigram" && d.pair_buckets > 0) {
    MI_TRY(dense());
    MI_TRY(check_matrix(name, shape, ndim, d.pair_buckets + 1, W));
    MI_TRY(put_raw(e, e->pair_embed, d.pair_buckets + 1, W, W, data, on_device));
    e->pair_embed_seen = true;
    return MI_OK;
  }
  if (name == "side.embed" && d.side_dim > 0) {
    MI_TRY(dense());
    MI_TRY(check_matrix(name, shape, ndim, d.vocab_size, d.num_layers * d.side_dim));
    MI_TRY(put_raw(e, e->side_embed, d.vocab_size, d.num_layers * d.side_dim, d.num_layers * d.side_dim, data, on_device));
    e->side_embed_seen = true;
    return MI_OK;
  }
  for (int i = 0; i < d.num_layers; ++i) {
    ListLayer& l = e->list[i];
    const mi_layer_desc& m = l.d;
    const std::string p = "l" + std::to_string(i) + ".";
    if (d.side_dim > 0 && name == p + "side.gate") {
      MI_TRY(dense());
      MI_TRY(check_matrix(name, shape, ndim, d.side_dim, W));
      MI_TRY(put_raw(e, l.side_gate, d.side_dim, W, e->wp, data, on_device));
      l.side_gate_seen = true;
      return MI_OK;
    }
    if (d.side_dim > 0 && name == p + "side.proj") {
      MI_TRY(dense());
      MI_TRY(check_matrix(name, shape, ndim, W, d.side_dim));
      PlaceCall pc{}; pc.nb = 1; pc.ni = W; pc.nj = d.side_dim; pc.si = d.side_dim; pc.sj = 1; pc.di = 1; pc.dj = e->wp;
      MI_TRY(put_placed(e, l.side_proj_t, (size_t)d.side_dim * e->wp, data, (size_t)W * d.side_dim, on_device, pc));
      if (side_mfma_supported(d.act_dtype, d.side_dim, e->wp)) {
        const int dp = up(d.side_dim, 32);
        pc.di = dp; pc.dj = 1;
        MI_TRY(put_placed(e, l.side_proj_p, (size_t)e->wp * dp, data, (size_t)W * d.side_dim, on_device, pc));
      }
      l.side_proj_seen = true;
      return MI_OK;
    }
    if (m.ff_kind == MI_FF_MOE && m.ff > 0 && name == p + "mlp.router") {
      MI_TRY(dense());
      MI_TRY(check_matrix(name, shape, ndim, m.experts, W));
      MI_TRY(put_raw(e, l.router, m.experts, W, e->wp, data, on_device));
      l.router_seen = true;
      return MI_OK;
    }
    if (m.mixer != MI_MIXER_LATENT) continue;
    const bool uk = name == p + "mix.uk", uv = name == p + "mix.uv";
    if (!uk && !uv) continue;
    const int hd = uk ? m.dim : m.vdim, rank = m.kv_rank;
    MI_TRY(dense());
    MI_TRY(check_matrix(name, shape, ndim, m.heads * hd, rank));
    MI_TRY(put_raw(e, uk ? l.uk : l.uv, m.heads * hd, rank, rank, data, on_device));
    if (l.kdp > 0) {
      const size_t es = act_size(e);
      for (int h = 0; h < m.heads; ++h)
        MI_TRY(put_rect(e, l.ukv, uk ? h * l.kdp : m.heads * l.kdp + h * l.vdp, 0, hd, rank, (const char*)data + (size_t)h * hd * rank * es, on_device));
      if (uk && m.rot_dims > 0) {                      // ones that hand the rotated key part through to every head
        std::vector<char> one((size_t)m.rot_dims * m.rot_dims * es, 0);
        for (int j = 0; j < m.rot_dims; ++j) {
          const uint16_t v = d.act_dtype == MI_BF16 ? 0x3f80 : 0x3c00;
          std::memcpy(&one[((size_t)j * m.rot_dims + j) * es], &v, 2);
        }
        for (int h = 0; h < m.heads; ++h) MI_TRY(put_rect(e, l.ukv, h * l.kdp + m.dim, l.cp, m.rot_dims, m.rot_dims, one.data(), 0));
      }
      PlaceCall pc{}; pc.nb = m.heads; pc.ni = hd; pc.nj = rank; pc.sb = (size_t)hd * rank; pc.si = rank; pc.sj = 1;
      if (uk) {
        pc.db = (size_t)l.rp * l.kdp; pc.di = 1; pc.dj = l.kdp;
        MI_TRY(put_placed(e, l.uk_t, (size_t)m.heads * l.rp * l.kdp, data, (size_t)m.heads * hd * rank, on_device, pc));
      } else {
        pc.db = (size_t)hd * l.rp; pc.di = l.rp; pc.dj = 1;
        MI_TRY(put_placed(e, l.uv_p, (size_t)m.heads * hd * l.rp, data, (size_t)m.heads * hd * rank, on_device, pc));
      }
    }
    (uk ? l.uk_seen : l.uv_seen) = true;
    return MI_OK;
  }
  return fail(MI_ERR_NOTFOUND, "unknown tensor: " + name);
}

int layers_finalize(mi_engine* e) {
  const mi_model_desc& d = e->d;
  std::string missing;
  each_vec(e, [&](Vec32& v) { if (v.n > 0 && !v.seen && !v.optional && missing.empty()) missing = v.name; });
  if (!missing.empty()) return fail(MI_ERR_NOTFOUND, missing + ": not set");
  if (!e->tok_embed_seen) return fail(MI_ERR_NOTFOUND, "embed: not set");
  if (d.side_dim > 0 && !e->side_embed_seen) return fail(MI_ERR_NOTFOUND, "side.embed: not set");
  if (d.pair_buckets > 0 && !e->pair_embed_seen) return fail(MI_ERR_NOTFOUND, "bigram: not set");
  for (int i = 0; i < d.num_layers; ++i) {
    ListLayer& l = e->list[i];
    const std::string p = "l" + std::to_string(i) + ".";
    if (d.side_dim > 0 && (!l.side_gate_seen || !l.side_proj_seen)) return fail(MI_ERR_NOTFOUND, p + "side.gate / side.proj: not set");
    if (l.d.mixer == MI_MIXER_LATENT && (!l.uk_seen || !l.uv_seen)) return fail(MI_ERR_NOTFOUND, p + "mix.uk / mix.uv: not set");
    MI_TRY(finalize_packed(e, l.in));
    MI_TRY(finalize_packed(e, l.out));
    if (l.lr.N > 0) MI_TRY(finalize_packed(e, l.lr));
    if (l.uq.N > 0) MI_TRY(finalize_packed(e, l.uq));
    if (l.d.ff_kind == MI_FF_DENSE && l.ffp > 0) {
      MI_TRY(finalize_packed(e, l.gu));
      MI_TRY(finalize_packed(e, l.dn));
      (void)ensure_gu8(e, l.gu.f, l.ffp);
    }
    if (l.d.mixer == MI_MIXER_LATENT && l.kdp > 0) MI_TRY(finalize_packed(e, l.ukv));
    if (l.d.ff_kind == MI_FF_MOE && l.d.ff > 0) {
      if (!l.router_seen) return fail(MI_ERR_NOTFOUND, p + "mlp.router: not set");
      MI_TRY(finalize_packed(e, l.gu));
      MI_TRY(finalize_packed(e, l.dn));
      if (l.sffp > 0) { MI_TRY(finalize_packed(e, l.sgu)); MI_TRY(finalize_packed(e, l.sdn)); }
    }
  }
  MI_TRY(finalize_packed(e, e->list_head));
  MI_HIP(hipStreamSynchronize(e->stream));
  return MI_OK;
}

void layers_free(mi_engine* e) {
  if (!e->layered) return;
  each_vec(e, [](Vec32& v) { hipFree(v.p); v.p = nullptr; });
  for (auto& l : e->list) {
    for (PackedLinear* L : {&l.in, &l.lr, &l.uq, &l.out, &l.ukv, &l.gu, &l.dn, &l.sgu, &l.sdn}) free_packed(*L);
    hipFree(l.decay); hipFree(l.log2_decay);
    hipFree(l.slopes); hipFree(l.router); hipFree(l.low_a); hipFree(l.low_g);
    hipFree(l.uk); hipFree(l.uv); hipFree(l.uk_t); hipFree(l.uv_p); hipFree(l.side_gate); hipFree(l.side_proj_t); hipFree(l.side_proj_p);
  }
  free_packed(e->list_head);
  for (auto& t : e->rot_tabs) hipFree(t.p);
  for (void* p : {e->tok_embed, e->side_embed, e->pair_embed, e->low, e->qc, e->qfull, (void*)e->light_ws, (void*)e->light_ctr, (void*)e->dl_q, (void*)e->d_freq, (void*)e->x32, e->hn, e->proj, e->cat, (void*)e->scan32, (void*)e->gate32,
                  e->lq, (void*)e->lat_part, e->lat_m, e->lat_x, e->lat_kv, (void*)e->dl_w, (void*)e->dl_p, (void*)e->dl_k, (void*)e->dl_f, (void*)e->d_meta, (void*)e->d_gather_list, e->head_x,
                  (void*)e->y32, e->v_first, (void*)e->moe_ids, (void*)e->moe_wts, e->moe_mid, e->moe_out, (void*)e->moe_plan, (void*)e->moe_counts, (void*)e->gqa_part, (void*)e->gqa_ctr}) hipFree(p);
}

// element offsets of the arenas (latents, keys, values) for `tokens` token places, byte offsets of the recurrent state for kv->B rows
int layers_kv_plan(mi_engine* e, mi_kv* kv) {
  const size_t es = dtype_size(kv->dtype);
  kv->arenas.clear(); kv->state_off.clear(); kv->ring_off.clear();
  const size_t tokens = kv->paged ? ((size_t)kv->nblocks << kv->bs_shift) : (size_t)kv->B * kv->cap;
  size_t at = 0, sb = 0;
  for (const LayerRun& r : e->runs) {
    const ListLayer& l = e->list[r.layer];
    auto arena = [&](int heads, int width) { kv->arenas.push_back(KvArena{at, heads, width}); at += tokens * heads * width; };
    if (r.lat >= 0) arena(1, l.rp);
    if (r.k >= 0) { arena(l.d.kv_heads, l.kdp); arena(l.d.kv_heads, l.vdp); }
    if (r.state >= 0) {
      const mi_layer_desc& m = l.d;
      kv->state_off.push_back(sb);
      sb += ((size_t)kv->B * m.heads * (m.mixer == MI_MIXER_LIGHTNING ? l.sd : m.dim) * m.vdim * sizeof(float) + 255) & ~(size_t)255;
      kv->ring_off.push_back(sb);
      if (m.mixer == MI_MIXER_DELTA) sb += ((size_t)kv->B * m.conv * (2 * m.kv_heads * m.dim + m.heads * m.vdim) * es + 255) & ~(size_t)255;
    }
  }
  if (e->d.pair_buckets > 0) sb += (size_t)kv->B * sizeof(int32_t);        // (the rows' last tokens stand at the end)
  kv->list_bytes = std::max<size_t>(16, at * es);
  kv->state_bytes = std::max<size_t>(16, sb);
  return MI_OK;
}

void layers_kv_bind(mi_engine* e, mi_kv* kv) {
  if (e->d.pair_buckets > 0) kv->d_prev = (int32_t*)(kv->state + kv->state_bytes) - kv->B;
}

int layers_ensure_workspace(mi_engine* e, size_t rows) {
  if (rows <= e->lw_rows) return MI_OK;
  MI_HIP(hipStreamSynchronize(e->stream));
  size_t n_in = 16, n_cat = 16, n_scan = 4, n_heads = 1, n_lq = 4, n_pick = 0, n_mid = 0, n_out = 0, n_plan = 0, n_count = 0, n_low = 0, n_qc = 0, n_q = 0;
  for (auto& l : e->list) {
    n_in = std::max(n_in, (size_t)l.in.N);
    n_cat = std::max(n_cat, (size_t)l.n_cat);
    if (l.d.mixer == MI_MIXER_DELTA) {
      n_scan = std::max(n_scan, (size_t)2 * l.d.kv_heads * l.d.dim + (size_t)l.d.heads * l.d.vdim + (l.d.decay_rank > 0 ? (size_t)l.d.heads * l.d.dim : 0));
      n_low = std::max(n_low, (size_t)l.lr.N);
      n_heads = std::max(n_heads, (size_t)l.d.heads);
    } else if (l.d.mixer == MI_MIXER_LIGHTNING) n_scan = std::max(n_scan, (size_t)l.d.heads * l.d.vdim);
    else n_lq = std::max(n_lq, (size_t)l.d.heads * (l.d.mixer == MI_MIXER_GQA ? l.kdp : l.rp));
    n_qc = std::max(n_qc, (size_t)l.qr);
    n_q = std::max(n_q, (size_t)l.uq.N);
    if (l.d.ff_kind == MI_FF_DENSE && l.ffp > 0) n_cat = std::max(n_cat, (size_t)l.ffp);      // (the mixer's output is done with by then)
    if (l.d.ff_kind == MI_FF_MOE && l.d.ff > 0) {
      const size_t slots = (size_t)l.d.top + (l.sffp > 0 ? 1 : 0);
      n_pick = std::max(n_pick, (size_t)l.d.top);
      n_mid = std::max(n_mid, slots * std::max(l.ffp, l.sffp));
      n_out = std::max(n_out, slots * e->wp);
      const RouteArgs r{l.d.experts, l.d.top, l.d.groups, l.d.keep, nullptr};
      n_plan = std::max(n_plan, moe_plan_ints((int)rows, r, l.sffp > 0 ? 1 : 0));
      n_count = std::max(n_count, moe_count_ints((int)rows, r));
    }
  }
  const size_t n_y = e->d.block_form == MI_BLOCK_PARALLEL ? 0 : e->wp;
  n_scan = up((int)n_scan, 4);
  e->scan_ld = (int)n_scan; e->gate_ld = (int)(4 * n_heads);
  const size_t es = act_size(e);
  struct B { void** p; size_t n; } bufs[] = {
      {(void**)&e->x32, rows * e->streams * e->wp * sizeof(float)}, {&e->hn, rows * e->wp * es}, {&e->proj, rows * n_in * es}, {&e->cat, rows * n_cat * es},
      {(void**)&e->scan32, rows * n_scan * sizeof(float)}, {(void**)&e->gate32, rows * 4 * n_heads * sizeof(float)},
      {&e->lq, rows * n_lq * sizeof(float)}, {&e->low, rows * n_low * es}, {&e->qc, rows * n_qc * es}, {&e->qfull, rows * n_q * es},
      {(void**)&e->y32, rows * n_y * sizeof(float)}, {&e->v_first, rows * (size_t)e->n_vfirst * es}, {(void**)&e->moe_ids, rows * n_pick * sizeof(int32_t)},
      {(void**)&e->moe_wts, rows * n_pick * sizeof(float)}, {&e->moe_mid, rows * n_mid * es}, {&e->moe_out, rows * n_out * es},
      {(void**)&e->moe_plan, n_plan * sizeof(int32_t)}, {(void**)&e->moe_counts, n_count * sizeof(int32_t)}};
  e->lw_rows = 0;
  for (auto& b : bufs) {
    hipFree(*b.p); *b.p = nullptr;
    if (b.n == 0) continue;
    MI_HIP(hipMalloc(b.p, b.n));
    MI_HIP(hipMemsetAsync(*b.p, 0, b.n, e->stream));      // (padding columns are multiplied by zero weights: they must be finite)
  }
  e->lw_rows = rows;
  return MI_OK;
}

int forward_segments(mi_engine* e, mi_kv* kv, const int32_t* rows, const int32_t* lens, int n, const int32_t* out_idx, int n_out) {
  const mi_model_desc& d = e->d;
  hipStream_t st = e->stream;
  const size_t es = act_size(e);
  const int act = d.act_dtype;
  for (int i = 0; i < n; ++i)
    if (kv->h_off[rows[i]] + lens[i] > kv->cap || kv->h_off[rows[i]] + lens[i] > d.max_positions)
      return fail(MI_ERR_INVALID, "forward: KV capacity / max_positions exceeded (call mi_kv_reserve)");
  for (int i = 0; i < n; ++i) MI_TRY(kv_ensure_blocks(kv, rows[i], kv->h_off[rows[i]] + lens[i]));
  MI_TRY(kv_upload_table(kv, st));
  Tables tb;
  MI_TRY(build_tables(e, kv, rows, lens, n, tb));
  const SegTables& t = tb.t;
  const int R = t.R;
  if (e->resid_out != nullptr && (int64_t)R * d.hidden_size * (int64_t)e->runs.size() > e->resid_cap)
    return fail(MI_ERR_INVALID, "residual capture: buffer too small for this pass");
  e->cur_L = t.nd == n ? 1 : 2;
  e->sq_valid = false;
  const int nstride = d.norm_kind == MI_NORM_SCALAR ? 0 : 1;
  const int32_t* tok = e->tok_src ? e->tok_src : e->d_tokens;
  const bool post = d.block_form == MI_BLOCK_POST_NORM, pre = d.block_form == MI_BLOCK_PRE_NORM, both = d.block_form == MI_BLOCK_SANDWICH;
  const int n_runs = (int)e->runs.size();
  auto norm_of = [&](int ri) {
    if (post) return RowNormW{nullptr, 0, 0.f};                // (no norm in front of a sublayer)
    const Vec32& v = ri < n_runs ? e->list[e->runs[ri].layer].norm : e->list_final_norm;
    return RowNormW{v.p, nstride, d.rms_norm_eps};
  };
  auto in_of = [&](int ri) { return d.streams > 0 && ri < n_runs ? e->list[e->runs[ri].layer].hc_in[0].p : nullptr; };
  { Prof pr(e, "embed");
    EmbedPosCall c{t, tok, e->tok_embed, e->d_freq, d.vocab_size, d.hidden_size, e->wp, norm_of(0), e->x32, e->hn, act};
    c.scale = d.embed_scale == 0.f ? 1.0f : d.embed_scale;
    c.pair = PairEmbed{e->pair_embed, d.pair_buckets, d.pair_mul_prev, d.pair_mul_cur, kv->d_prev};
    c.streams = d.streams; c.in = in_of(0);
    MI_TRY(launch_embed_pos(c, st)); }
  // pre-norm blocks: sublayer q of a layer has left y32; `in` and `norm` are the next sublayer's
  auto stream_norm = [&](const ListLayer& l, int q, const float* in, RowNormW norm, bool last) -> int {
    StreamNormCall c{R, e->y32, d.streams, l.hc_mix[q].p, l.hc_out[q].p, in, d.residual_mult == 0.f ? 1.0f : d.residual_mult, norm,
                     d.hidden_size, e->wp, e->x32, e->hn, last && e->resid_out == nullptr ? 0 : 1, act};
    Prof pr(e, "stream_norm");
    return launch_stream_norm(c, st);
  };
  for (int ri = 0; ri < n_runs; ++ri) {
    const LayerRun& run = e->runs[ri];
    const int li = run.layer;
    ListLayer& l = e->list[li];
    const mi_layer_desc& m = l.d;
    GemvCall ci; ci.x = e->hn; ci.ldx = e->wp; ci.act = act; ci.epi = EPI_STORE; ci.out = e->proj; ci.ldo = l.in.N;
    if (m.mixer == MI_MIXER_LIGHTNING) ci.silu_cols = l.o_g;             // (q, k and v stand in front of the gate)
    MI_TRY(gemv_rows(e, l.in.f, ci, R, es, es, "gemv_in"));
    const PolyNormArgs ff{post || pre || both ? 0 : m.ff, l.o_up, l.o_ff, l.act.p, d.rms_norm_eps};
    if (m.mixer == MI_MIXER_DELTA) {
      const bool channel = m.decay_rank > 0;
      if (l.lr.N > 0 && (l.low_a == nullptr || t.nc > 0)) {
        const char* x = (const char*)e->proj + (size_t)l.o_lr * es;
        const LowRankCall lc{l.lr.f.W, l.o_g, up(m.decay_rank, 64), x, l.in.N, R, e->low, l.lr.N, act};
        if (R >= 256 && m.decay_rank > 0 && up(m.gate_rank, 64) == lc.k && low_rank_supported(lc)) {
          Prof pr(e, "gemv_low");
          MI_TRY(launch_low_rank(lc, st));
        } else {
          GemvCall cl; cl.x = x; cl.ldx = l.in.N; cl.act = act; cl.epi = EPI_STORE; cl.out = e->low; cl.ldo = l.lr.N;
          MI_TRY(gemv_rows(e, l.lr.f, cl, R, es, es, "gemv_low"));
        }
      }
      DeltaCall c{};
      c.t = t; c.H = m.heads; c.G = m.kv_heads; c.d = m.dim; c.e = m.vdim; c.taps = m.conv;
      c.proj = e->proj; c.ldp = l.in.N;
      c.o_q = l.o_q; c.o_k = l.o_k; c.o_v = l.o_v; c.o_g = l.o_g; c.o_b = l.o_b; c.o_a = l.o_a;
      c.ap = channel ? e->low : e->proj; c.ldap = channel ? l.lr.N : l.in.N;
      c.gp = m.gate_rank > 0 ? e->low : e->proj; c.ldgp = m.gate_rank > 0 ? l.lr.N : l.in.N;
      c.channel = channel; c.gate_act = m.out_gate;
      c.low_a = l.low_a; c.low_g = l.low_g; c.ld_a = up(m.decay_rank, 8); c.ld_gt = up(m.gate_rank, 8); c.in_a = l.o_lr; c.in_g = l.o_lrg;
      c.conv_q = l.conv_q.p; c.conv_k = l.conv_k.p; c.conv_v = l.conv_v.p;
      c.A_log = l.A_log.p; c.dt_bias = l.dt_bias.p; c.head_norm = l.head_norm.p;
      c.scale = m.scale; c.unit_eps = m.unit_eps; c.eps = d.rms_norm_eps;
      c.state = (float*)(kv->state + kv->state_off[run.state]);
      c.ring = kv->state + kv->ring_off[run.state];
      c.scan = e->scan32; c.lds = e->scan_ld; c.gate = e->gate32; c.ldg = e->gate_ld;
      c.cat = e->cat; c.ldc = l.n_cat; c.ff = ff; c.act = act;
      const int cp = delta_chunk_pad(m.heads, m.dim, m.vdim, m.conv);
      if (cp > 0 && tb.maxlen >= DELTA_CHUNK_FROM && std::max((size_t)R * e->scan_ld, (size_t)R * m.heads * std::max(cp, DELTA_CHUNK)) < ((size_t)1 << 30)) {
        MI_TRY(grow(e, (void**)&e->dl_w, &e->dl_w_cap, (size_t)R * m.heads * cp * sizeof(float)));
        MI_TRY(grow(e, (void**)&e->dl_p, &e->dl_p_cap, (size_t)R * m.heads * DELTA_CHUNK * sizeof(float)));
        MI_TRY(grow(e, (void**)&e->dl_k, &e->dl_k_cap, (size_t)t.nct * (channel ? m.heads : m.kv_heads) * cp * DELTA_CHUNK * sizeof(float)));
        MI_TRY(grow(e, (void**)&e->dl_f, &e->dl_f_cap, (size_t)t.nct * m.heads * (channel ? cp : DELTA_FAC) * sizeof(float)));
        if (channel) MI_TRY(grow(e, (void**)&e->dl_q, &e->dl_q_cap, (size_t)R * m.heads * cp * sizeof(float)));
        c.wm = e->dl_w; c.pm = e->dl_p; c.kt = e->dl_k; c.fac = e->dl_f; c.qm = e->dl_q;
      }
      Prof pr(e, "delta");
      MI_TRY(launch_delta(c, st));
    } else if (m.mixer == MI_MIXER_GQA) {
      MI_TRY(run_gqa(e, kv, l, run, tb, rows, lens, n));
    } else if (m.mixer == MI_MIXER_LIGHTNING) {
      MI_TRY(run_lightning(e, kv, l, run, tb));
    } else {
      LatentCall c{};
      int li_src = run.lat;                // (a layer that reads another's latents stands in a stack without loops: run = layer)
      if (li_src < 0) li_src = e->runs[l.src].lat;
      c.t = t;
      c.s = AttnShape{1, 1, m.heads, 1, l.rp, act, kv->dtype, RND_NONE, kv->cap, nullptr, nullptr, 0, 0};
      kv_shape(kv, c.s);
      c.H = m.heads; c.dim = m.dim; c.vdim = m.vdim; c.rank = m.kv_rank; c.rp = l.rp; c.kdp = l.kdp; c.vdp = l.vdp;
      c.rot = m.rot_dims; c.cp = l.cp; c.pairs = m.rot_pairs; c.rot_tab = l.rot_tab;
      c.proj = e->proj; c.ldp = l.in.N; c.o_g = l.o_g; c.o_c = l.o_c;
      c.q = m.q_rank > 0 ? e->qfull : (const char*)e->proj + (size_t)l.o_q * es; c.ldq = m.q_rank > 0 ? l.uq.N : l.in.N;
      c.q_rank = m.q_rank; c.ldqc = l.qr; c.q_norm = l.dq_norm.p; c.qc = e->qc; c.o_qc = l.o_qc;
      c.c_norm = l.c_norm.p; c.eps = d.rms_norm_eps;
      c.cache = (char*)kv->k + kv->arenas[li_src].off * dtype_size(kv->dtype);
      c.uk = l.uk; c.uv = l.uv; c.uk_t = l.uk_t; c.uv_p = l.uv_p; c.scale = m.scale;
      c.lq = e->lq; c.nsplit = 1;
      c.cat = e->cat; c.ldc = l.n_cat; c.ff = ff; c.act = act;
      MI_TRY(run_latent(e, kv, l, tb, rows, lens, n, c));
    }
    GemvCall co; co.x = e->cat; co.ldx = l.n_cat; co.act = act; co.epi = EPI_RESID; co.out32 = 1; co.resid = e->x32; co.ldo = e->wp;
    if (post || pre || both) { co.epi = EPI_STORE; co.resid = nullptr; co.out = e->y32; }
    MI_TRY(gemv_rows(e, l.out.f, co, R, es, sizeof(float), "gemv_out"));
    // gate | up with the unit in the epilogue, down: y32
    auto dense_ff = [&]() -> int {
      GemvCall cg; cg.x = e->hn; cg.ldx = e->wp; cg.act = act; cg.epi = EPI_SWIGLU; cg.out = e->cat; cg.ldo = l.ffp; cg.pair_offset = l.ffp; cg.glu = l.glu;
      MI_TRY(gemv_rows(e, l.gu.f, cg, R, es, es, "gemv_gate_up"));
      GemvCall cd; cd.x = e->cat; cd.ldx = l.ffp; cd.act = act; cd.epi = EPI_STORE; cd.out32 = 1; cd.out = e->y32; cd.ldo = e->wp;
      return gemv_rows(e, l.dn.f, cd, R, es, sizeof(float), "gemv_down");
    };
    if (post || both) {
      PostNormCall pn{};
      pn.rows = R; pn.y = e->y32; pn.kind = d.norm_kind; pn.eps = d.rms_norm_eps; pn.norm = both ? PostNormW{l.norm_out.p, nullptr, nstride} : PostNormW{l.norm.p, l.norm_b.p, nstride};
      pn.width = d.hidden_size; pn.ld = e->wp; pn.x = e->x32; pn.h = e->hn; pn.act = act;
      const PostNormW last{e->list_final_norm.p, e->list_final_norm_b.p, nstride};
      const bool end = ri + 1 == n_runs;
      if (both && m.ff > 0) pn.next = PostNormW{l.norm2.p, nullptr, nstride};
      if (m.ff > 0 && m.ff_kind == MI_FF_DENSE) {
        { Prof pr(e, "post_norm"); MI_TRY(launch_post_norm(pn, st)); }
        MI_TRY(dense_ff());
      } else if (m.ff > 0) {
        const MoeCall mc = moe_call(e, l, R);
        const bool fused = route_fused(act, R, m.experts);
        pn.r = mc.r; pn.ids = mc.ids; pn.wts = mc.wts;
        pn.router = fused ? l.router : nullptr;
        if (!fused) { pn.clear = mc.counts; pn.n_clear = m.experts; }
        { Prof pr(e, "post_norm"); MI_TRY(launch_post_norm(pn, st)); }
        if (!fused) { Prof pr(e, "moe_route"); MI_TRY(launch_route(mc, st)); }
        { Prof pr(e, "moe_plan"); MI_TRY(launch_moe_plan(mc, st)); }
        { Prof pr(e, "moe_up"); MI_TRY(launch_moe_up(mc, st)); }
        { Prof pr(e, "moe_down"); MI_TRY(launch_moe_down(mc, st)); }
        pn.y = nullptr; pn.parts = mc.out; pn.part_w = mc.wts; pn.top = m.top; pn.shared = l.sffp > 0 ? 1 : 0; pn.router = nullptr; pn.clear = nullptr;
      }
      if (m.ff > 0) pn.norm = both ? PostNormW{l.norm2_out.p, nullptr, nstride} : PostNormW{l.norm2.p, l.norm2_b.p, nstride};
      pn.next = end ? last : (both ? PostNormW{e->list[e->runs[ri + 1].layer].norm.p, nullptr, nstride} : PostNormW{nullptr, nullptr, 0});
      Prof pr(e, m.ff > 0 ? "post_norm2" : "post_norm");
      MI_TRY(launch_post_norm(pn, st));
    } else if (pre) {
      int q = 0;
      if (m.ff > 0) {
        MI_TRY(stream_norm(l, 0, l.hc_in[1].p, RowNormW{l.norm2.p, nstride, d.rms_norm_eps}, false));
        MI_TRY(dense_ff());
        q = 1;
      }
      MI_TRY(stream_norm(l, q, in_of(ri + 1), norm_of(ri + 1), ri + 1 == n_runs));
    } else { Prof pr(e, "side");
      SideNormCall c{R, tok, e->side_embed, d.num_layers * d.side_dim, li * d.side_dim, d.vocab_size, l.side_gate, l.side_proj_t, l.side_proj_p,
                     l.side_norm.p, d.rms_norm_eps, d.side_dim, d.hidden_size, e->wp, norm_of(ri + 1), e->x32, e->hn, act};
      MI_TRY(launch_side_norm(c, st)); }
    if (e->resid_out != nullptr) {
      const float* x = e->x32;
      if (e->streams > 1) { MI_TRY(launch_stream_sum(e->x32, e->streams, R, e->wp, e->y32, st)); x = e->y32; }
      MI_HIP(hipMemcpy2DAsync(e->resid_out + (size_t)ri * R * d.hidden_size, d.hidden_size * sizeof(float), x, e->wp * sizeof(float),
                              d.hidden_size * sizeof(float), R, hipMemcpyDeviceToHost, st));
      MI_HIP(hipStreamSynchronize(st));
    }
  }
  if (n_out > 0) {
    const void* hx = e->hn;
    bool all = n_out == R;
    for (int i = 0; i < n_out && all; ++i) all = out_idx[i] == i;
    if (!all) {                   // normed rows of the wanted positions, compacted (proj is free by now and holds at least as many bytes per row)
      MI_TRY(grow(e, (void**)&e->d_gather_list, &e->d_gather_list_cap, (size_t)n_out * sizeof(int32_t)));
      MI_HIP(hipMemcpyAsync(e->d_gather_list, out_idx, n_out * sizeof(int32_t), hipMemcpyHostToDevice, st));
      MI_TRY(grow(e, &e->head_x, &e->head_x_cap, (size_t)n_out * e->wp * es));
      MI_TRY(launch_gather_rows(e->hn, (size_t)e->wp * es, e->d_gather_list, n_out, e->head_x, st));
      hx = e->head_x;
    }
    GemvCall c; c.x = hx; c.ldx = e->wp; c.act = act; c.epi = EPI_STORE; c.out32 = 1; c.out = e->logits; c.ldo = d.vocab_size;
    const int keep = e->cur_L;
    e->cur_L = n_out <= 96 ? 1 : 2;          // (the few sampled rows of a step: the decode step's kernels)
    const int rc = gemv_rows(e, e->list_head.f, c, n_out, es, sizeof(float), "gemv_head");
    e->cur_L = keep;
    MI_TRY(rc);
    Prof pr(e, "logit_cap");
    MI_TRY(launch_logit_cap(e->logits, (size_t)n_out * d.vocab_size, d.logit_scale == 0.f ? 1.0f : d.logit_scale, d.logit_softcap, st));
  }
  MI_TRY(launch_advance_segments(t, kv->d_off, tok, kv->d_prev, st));
  for (int i = 0; i < n; ++i) kv->h_off[rows[i]] += lens[i];
  return MI_OK;
}

}  // namespace mi

extern "C" {

int mi_engine_create_layers(const mi_model_desc* desc, const mi_layer_desc* layers, int n_layers, int device, mi_engine** out) {
  if (!desc || !layers || !out) return fail(MI_ERR_INVALID, "null argument");
  if (desc->struct_size != sizeof(mi_model_desc)) return fail(MI_ERR_INVALID, "mi_model_desc.struct_size does not match this library");
  const mi_model_desc& d = *desc;
  if (d.arch != MI_ARCH_LAYERS) return fail(MI_ERR_INVALID, "mi_engine_create_layers: desc.arch must be MI_ARCH_LAYERS");
  if (d.hidden_size <= 0 || d.vocab_size <= 0 || d.max_positions <= 0 || d.side_dim < 0 || n_layers < 1 || n_layers != d.num_layers)
    return fail(MI_ERR_INVALID, "model dimensions must be positive");
  if (d.act_dtype != MI_F32 && d.act_dtype != MI_BF16 && d.act_dtype != MI_F16) return fail(MI_ERR_INVALID, "bad act_dtype");
  if (d.quant_bits != 0) return fail(MI_ERR_UNSUPPORTED, "layer-list models: no quantised weights");
  if (d.position != MI_POS_NONE && d.position != MI_POS_SINUSOIDAL) return fail(MI_ERR_UNSUPPORTED, "unknown position encoding");
  if (d.block_form != MI_BLOCK_PARALLEL && d.block_form != MI_BLOCK_POST_NORM && d.block_form != MI_BLOCK_PRE_NORM &&
      d.block_form != MI_BLOCK_SANDWICH)
    return fail(MI_ERR_UNSUPPORTED, "unknown block form");
  const bool post = d.block_form == MI_BLOCK_POST_NORM, pre = d.block_form == MI_BLOCK_PRE_NORM, both = d.block_form == MI_BLOCK_SANDWICH;
  if (d.norm_kind != MI_NORM_VECTOR && d.norm_kind != MI_NORM_SCALAR && !(post && d.norm_kind == MI_NORM_LAYER)) return fail(MI_ERR_UNSUPPORTED, "unknown norm");
  if ((post || pre || both) && d.side_dim > 0) return fail(MI_ERR_UNSUPPORTED, "per-layer token input: parallel blocks only");
  if (d.streams < 0 || d.streams > MAX_STREAMS) return fail(MI_ERR_INVALID, "streams must be in [0, 16]");
  if (d.streams > 0 && !pre) return fail(MI_ERR_UNSUPPORTED, "hyper-connections: pre-norm blocks only");
  if (d.pair_buckets < 0 || (d.pair_buckets > 0 && (d.pair_mul_prev < 0 || d.pair_mul_prev >= d.pair_buckets || d.pair_mul_cur < 0 || d.pair_mul_cur >= d.pair_buckets)))
    return fail(MI_ERR_INVALID, "pair embedding: multipliers must be in [0, buckets)");
  if (d.loop_stop < 0 || (d.loop_stop > 0 && (d.loop_start < 0 || d.loop_start >= d.loop_stop || d.loop_stop > d.num_layers || d.loop_times < 0)))
    return fail(MI_ERR_INVALID, "loop: not a range of the layers");
  int ndev = 0;
  if (hipGetDeviceCount(&ndev) != hipSuccess || ndev <= 0)
    return fail(MI_ERR_RUNTIME, "no HIP device available (this library has no CPU backend)");
  if (device < 0 || device >= ndev) return fail(MI_ERR_INVALID, "bad device index");
  MI_HIP(hipSetDevice(device));
  mi_engine* e = new mi_engine();
  e->d = d; e->device = device;
  if (hipStreamCreateWithFlags(&e->stream, hipStreamNonBlocking) != hipSuccess) { delete e; return fail(MI_ERR_RUNTIME, "hipStreamCreate failed"); }
  const int rc = init_layers(e, layers);
  if (rc != MI_OK) { mi_engine_destroy(e); return rc; }
  *out = e;
  return MI_OK;
}

int mi_debug_residual(mi_engine* e, float* out, int64_t capacity_floats) {
  if (!e) return fail(MI_ERR_INVALID, "null engine");
  if (!e->layered) return fail(MI_ERR_UNSUPPORTED, "residual capture: layer-list models only");
  e->resid_out = out; e->resid_cap = capacity_floats;
  return MI_OK;
}

}  // extern "C"
