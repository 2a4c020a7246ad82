// gqa.hip -- grouped-query attention (layer-list models).  q and k are divided by their root mean square and their first
// coordinates rotated by the position (or first rotated and then divided), head h scores  softcap tanh(q.k scale / softcap) - slope_h (i - j)  over the keys j <= i of i's
// own chunk of positions (or of a window behind i and the kept first tokens of the sequence), the denominator of the softmax also
// contains exp(sink_h), the values are mixed with an earlier layer's of the same token before they are cached, and the output is
// multiplied with sigmoid(gate), element by element or head by head.  Keys and values may be an earlier layer's: then nothing is
// appended.  Each of these is a parameter that can be off.
// A rotation keeps the length of a pair up to the table's gain, so the mean square behind it is that of the plain coordinates with the
// rotated ones weighted by the gain squared (rot_gain2): both orders of norm and rotation run as norm, then rotation.
//
//   gqa_pre        norms, rotation, value mix and append of every token of the longer segments (generic form: of all tokens)
//   gqa_generic    any size and dtype: one workgroup per (token, query head), float32 arithmetic
//   gqa_decode     16-bit caches, one-token segments: norms, rotation, append, split-KV attention, combine and gate in ONE launch; the query
//                  heads of a group are the columns of the MFMAs and share every key and value that is read
//   gqa_prefill    16-bit caches, longer segments: flash attention over the paged cache, tiles of 64 or 128 queries of one head
// Only the key blocks that a tile's chunks or windows reach are walked, and those of the kept tokens.
#include <algorithm>
#include <type_traits>

#include "layer_rows.h"

namespace mi {

namespace {

using namespace rows;

typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef _Float16 f16x8 __attribute__((ext_vector_type(8)));
constexpr float LOG2E = 1.4426950408889634f;

__device__ __forceinline__ size_t cache_at(const AttnShape& s, int row, int head, int key) {
  return s.btab ? kv_elem<true>(s, row, head, key) : kv_elem<false>(s, row, head, key);
}
// the query at `pos` sees the keys [first_seen, pos] and [0, keep)
__device__ __forceinline__ int first_seen(const GqaCall& c, int pos) {
  return c.window > 0 ? max(0, pos - c.window + 1) : (c.chunk > 0 ? pos / c.chunk * c.chunk : 0);
}

// weight of coordinate k in the mean square
__device__ __forceinline__ float square_weight(const GqaCall& c, int k) { return k < c.rot ? c.rot_gain2 : 1.f; }
// where head h's gates begin, and the one of its element d
__device__ __forceinline__ int gate_at(const GqaCall& c, int h, int d) { return c.gate_head ? h : h * c.vdim + d; }

// What the rotation of the N coordinates k .. k + N - 1 of a head needs besides themselves: their partners (as projected, and the
// partners' norm weights), cosine and sine.
template <int N>
struct Rot { float v[N], w[N], c[N], s[N]; };
template <typename T, int N>
__device__ __forceinline__ void load_rot(const GqaCall& c, const T* src, const float* w, int k, int pos, Rot<N>& r) {
  const int half = c.rot >> 1;
  const float2* tab = c.rot_tab + (size_t)pos * half;
#pragma unroll
  for (int i = 0; i < N; ++i) { r.v[i] = 0.f; r.w[i] = 0.f; r.c[i] = 1.f; r.s[i] = 0.f; }
  if (k >= c.rot) return;
  typedef T tv __attribute__((ext_vector_type(N)));
  if (c.pairs) {
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const int j = k + i;
      if (j >= c.rot) continue;
      const RotAt a = rot_at(j, c.rot, 1);
      const float2 cs = tab[a.f];
      r.v[i] = to_f32(src[a.partner]); r.w[i] = w[a.partner]; r.c[i] = cs.x; r.s[i] = a.sign * cs.y;
    }
    return;
  }
  if (half % N == 0 && k % N == 0) {                 // (the N coordinates lie in one half)
    const int p = k < half ? k + half : k - half, f = k < half ? k : k - half;
    const bool aligned = ((uintptr_t)(src + p) & (N * sizeof(T) - 1)) == 0;
    if (aligned) {
      const tv x = *(const tv*)(src + p);
#pragma unroll
      for (int i = 0; i < N; ++i) r.v[i] = to_f32(x[i]);
    } else {
#pragma unroll
      for (int i = 0; i < N; ++i) r.v[i] = to_f32(src[p + i]);
    }
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const float2 cs = tab[f + i];
      r.w[i] = w[p + i]; r.c[i] = cs.x; r.s[i] = k < half ? -cs.y : cs.y;
    }
    return;
  }
#pragma unroll
  for (int i = 0; i < N; ++i) {
    const int j = k + i;
    if (j >= c.rot) continue;
    const RotAt a = rot_at(j, c.rot, 0);
    const float2 cs = tab[a.f];
    r.v[i] = to_f32(src[a.partner]); r.w[i] = w[a.partner]; r.c[i] = cs.x; r.s[i] = a.sign * cs.y;
  }
}
// v: the normed coordinates, rs: the head's reciprocal root mean square
template <int N>
__device__ __forceinline__ void rotate(const Rot<N>& r, float rs, float (&v)[N]) {
#pragma unroll
  for (int i = 0; i < N; ++i) v[i] = v[i] * r.c[i] + r.v[i] * rs * r.w[i] * r.s[i];
}

// ---- norms, value mix, append ----------------------------------------------------------------------------------------
// grid R.  VEC: head sizes are multiples of 8 up to 128 (coordinates rotated in halves: of 16), 16 lanes per head; otherwise a wave per head.
template <typename T, bool VEC, bool ROT>
__global__ __launch_bounds__(256) void gqa_pre_kernel(GqaCall c) {
  const int r = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const TokenAt at = token_at(c.t, r);
  if (!c.all_tokens && c.t.len[at.seg] == 1) return;           // (gqa_decode does its own)
  const T* pr = (const T*)c.proj + (size_t)r * c.ldp;
  const float lam = c.v_mix != nullptr ? *c.v_mix : 0.f;
  const int nh = c.H + (c.shared ? 0 : 2 * c.G);
  if constexpr (VEC) {
    const int g = lane >> 4, l = lane & 15;
    for (int h0 = wave * 4; h0 < nh; h0 += 16) {
      const int h = h0 + g;
      if (h >= nh) continue;                                    // (whole groups of 16 lanes)
      const int kind = h < c.H ? 0 : (h < c.H + c.G ? 1 : 2), hh = kind == 0 ? h : (kind == 1 ? h - c.H : h - c.H - c.G);
      const int n = kind == 2 ? c.vdim : c.dim, np = kind == 2 ? c.vdp : c.kdp, k = 8 * l;
      const T* src = pr + (kind == 0 ? c.o_q : (kind == 1 ? c.o_k : c.o_v)) + hh * n;
      float v[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] = 0.f;
      if (k < n) load8f<T>(src + k, v);
      if (kind < 2) {
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) ss += v[i] * v[i] * square_weight(c, k + i);
        const float rs = 1.0f / sqrtf(row16_sum(ss) / (float)n + c.eps);
        const float* w = kind == 0 ? c.q_norm : c.k_norm;
        if (k < n) {
#pragma unroll
          for (int i = 0; i < 8; ++i) v[i] *= rs * w[k + i];
        }
        if (ROT && c.pairs) {                                   // (the partners are this lane's)
          const float2* tab = c.rot_tab + (size_t)at.pos * (c.rot >> 1);
          float u[8];
#pragma unroll
          for (int i = 0; i < 8; ++i) u[i] = v[i];
#pragma unroll
          for (int i = 0; i < 8; ++i) {
            if (k + i >= c.rot) continue;
            const float2 cs = tab[(k + i) >> 1];
            v[i] = u[i] * cs.x + ((i & 1) ? u[i ^ 1] : -u[i ^ 1]) * cs.y;
          }
        } else if constexpr (ROT) {                             // (rot a multiple of 16: the partners are another lane's eight, normed)
          const int half = c.rot >> 1;
          const bool on = k < c.rot, low = k < half;
          const int with = on ? (low ? lane + half / 8 : lane - half / 8) : lane;
          const float2* tab = c.rot_tab + (size_t)at.pos * half + (on ? (low ? k : k - half) : 0);
#pragma unroll
          for (int i = 0; i < 8; ++i) {
            const float u = __shfl(v[i], with, 64);
            const float2 cs = tab[i];
            if (on) v[i] = v[i] * cs.x + (low ? -u : u) * cs.y;
          }
        }
      } else {
        const size_t fo = (size_t)r * c.G * c.vdim + hh * c.vdim + k;
        if (k < n && c.v_first_out != nullptr) store8f<T>((T*)c.v_first_out + fo, v);
        if (k < n && c.v_mix != nullptr) {
          float f[8];
          load8f<T>((const T*)c.v_first_in + fo, f);
#pragma unroll
          for (int i = 0; i < 8; ++i) v[i] = (1.0f - lam) * v[i] + lam * f[i];
        }
      }
      if (k < np) {
        T* dst = kind == 0 ? (T*)c.q + ((size_t)r * c.H + hh) * c.kdp
                           : (kind == 1 ? (T*)c.kcache + cache_at(c.sk, at.row, hh, at.pos) : (T*)c.vcache + cache_at(c.sv, at.row, hh, at.pos));
        store8f<T>(dst + k, v);
      }
    }
  } else {
    for (int h = wave; h < nh; h += 4) {
      const int kind = h < c.H ? 0 : (h < c.H + c.G ? 1 : 2), hh = kind == 0 ? h : (kind == 1 ? h - c.H : h - c.H - c.G);
      const int n = kind == 2 ? c.vdim : c.dim, np = kind == 2 ? c.vdp : c.kdp;
      const T* src = pr + (kind == 0 ? c.o_q : (kind == 1 ? c.o_k : c.o_v)) + hh * n;
      T* dst = kind == 0 ? (T*)c.q + ((size_t)r * c.H + hh) * c.kdp
                         : (kind == 1 ? (T*)c.kcache + cache_at(c.sk, at.row, hh, at.pos) : (T*)c.vcache + cache_at(c.sv, at.row, hh, at.pos));
      float rs = 1.0f;
      const float* w = kind == 0 ? c.q_norm : c.k_norm;
      if (kind < 2) {
        float ss = 0.f;
        for (int k = lane; k < n; k += 64) { const float v = to_f32(src[k]); ss += v * v * square_weight(c, k); }
        rs = 1.0f / sqrtf(wave_sum(ss) / (float)n + c.eps);
      }
      for (int k = lane; k < np; k += 64) {
        float v = k < n ? to_f32(src[k]) : 0.f;
        if (kind < 2) {
          if (k < n) v *= rs * w[k];
          if (ROT && k < c.rot) {
            Rot<1> ro;
            float one[1] = {v};
            load_rot<T, 1>(c, src, w, k, at.pos, ro);
            rotate<1>(ro, rs, one);
            v = one[0];
          }
        } else if (k < n) {
          const size_t fo = (size_t)r * c.G * c.vdim + hh * c.vdim + k;
          if (c.v_first_out != nullptr) ((T*)c.v_first_out)[fo] = from_f32<T>(v);
          if (c.v_mix != nullptr) v = (1.0f - lam) * v + lam * to_f32(((const T*)c.v_first_in)[fo]);
        }
        dst[k] = from_f32<T>(v);
      }
    }
  }
}

// ---- generic form ----------------------------------------------------------------------------------------------------
// grid (R, H), 4 waves: wave w takes keys w, w + 4, .. of the kept and the other visible ones; NR key / value elements per lane
template <typename T, int NR>
__global__ __launch_bounds__(256) void gqa_generic_kernel(GqaCall c) {
  extern __shared__ float sm[];                      // [4][vdp] sums
  __shared__ float ml[8];
  const int r = blockIdx.x, h = blockIdx.y, g = h / (c.H / c.G), lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const TokenAt at = token_at(c.t, r);
  const int lo = first_seen(c, at.pos), kept = min(c.keep, lo), n = kept + at.pos - lo + 1;      // visible keys, in order
  auto key_at = [&](int i) { i = min(i, n - 1); return i < kept ? i : lo + i - kept; };
  const T* qp = (const T*)c.q + ((size_t)r * c.H + h) * c.kdp;
  const float slope = c.slopes[h];
  float q[NR], o[NR], m = -INFINITY, l = 0.f;
#pragma unroll
  for (int i = 0; i < NR; ++i) { const int k = lane + 64 * i; q[i] = k < c.dim ? to_f32(qp[k]) : 0.f; o[i] = 0.f; }
  constexpr int U = NR <= 2 ? 4 : 2;                 // keys in flight
  for (int i0 = wave; i0 < n; i0 += 4 * U) {
    float x[U][NR], sc[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const T* p = (const T*)c.kcache + cache_at(c.sk, at.row, g, key_at(i0 + 4 * u));
      float a = 0.f;
#pragma unroll
      for (int i = 0; i < NR; ++i) { const int k = lane + 64 * i; if (k < c.dim) a = fmaf(q[i], to_f32(p[k]), a); }
      sc[u] = a;
      const T* pv = (const T*)c.vcache + cache_at(c.sv, at.row, g, key_at(i0 + 4 * u));
#pragma unroll
      for (int i = 0; i < NR; ++i) { const int k = lane + 64 * i; x[u][i] = k < c.vdim ? to_f32(pv[k]) : 0.f; }
    }
    float mx = m;
#pragma unroll
    for (int u = 0; u < U; ++u) {
      float s = wave_sum(sc[u]) * c.scale;
      if (c.softcap > 0.f) s = c.softcap * tanhf(s / c.softcap);
      sc[u] = s - slope * (float)(at.pos - key_at(i0 + 4 * u));
      if (i0 + 4 * u < n) mx = fmaxf(mx, sc[u]);
    }
    const float corr = expf(m - mx);                 // (the first key of the loop is visible: mx is finite)
    m = mx; l *= corr;
#pragma unroll
    for (int i = 0; i < NR; ++i) o[i] *= corr;
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const float p = i0 + 4 * u < n ? expf(sc[u] - m) : 0.f;
      l += p;
#pragma unroll
      for (int i = 0; i < NR; ++i) o[i] = fmaf(p, x[u][i], o[i]);
    }
  }
#pragma unroll
  for (int i = 0; i < NR; ++i) { const int k = lane + 64 * i; if (k < c.vdim) sm[wave * c.vdp + k] = o[i]; }
  if (lane == 0) { ml[wave] = m; ml[4 + wave] = l; }
  __syncthreads();
  float mx = fmaxf(fmaxf(ml[0], ml[1]), fmaxf(ml[2], ml[3]));
  if (c.sink != nullptr) mx = fmaxf(mx, c.sink[h]);
  float w[4], lt = c.sink != nullptr ? expf(c.sink[h] - mx) : 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) { w[i] = expf(ml[i] - mx); lt += w[i] * ml[4 + i]; }
  const T* gate = (const T*)c.proj + (size_t)r * c.ldp + max(c.o_g, 0);
  T* cat = (T*)c.cat + (size_t)r * c.ldc + h * c.vdim;
  for (int k = threadIdx.x; k < c.vdim; k += 256) {
    const float v = (w[0] * sm[k] + w[1] * sm[c.vdp + k] + w[2] * sm[2 * c.vdp + k] + w[3] * sm[3 * c.vdp + k]) / lt;
    cat[k] = from_f32<T>(c.o_g >= 0 ? v * sigmoid_f(to_f32(gate[gate_at(c, h, k)])) : v);
  }
}

// ---- matrix-core forms ------------------------------------------------------------------------------------------------
template <typename T>
__device__ __forceinline__ f32x4 mfma16(u32x4 a, u32x4 b, f32x4 c) {
  if constexpr (std::is_same<T, bf16>::value)
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
  else
    return __builtin_amdgcn_mfma_f32_16x16x32_f16(__builtin_bit_cast(f16x8, a), __builtin_bit_cast(f16x8, b), c, 0, 0, 0);
}

// two float32 values as hi + lo pairs of 16-bit values (softmax weights keep 32-bit accuracy through two MFMAs)
template <typename T>
__device__ __forceinline__ void split2(float a, float b, uint32_t& hi, uint32_t& lo) {
  typedef float f32x2 __attribute__((ext_vector_type(2)));
  typedef T tx2 __attribute__((ext_vector_type(2)));
  const tx2 h = __builtin_convertvector((f32x2{a, b}), tx2);
  const f32x2 back = __builtin_convertvector(h, f32x2);
  hi = __builtin_bit_cast(uint32_t, h);
  lo = __builtin_bit_cast(uint32_t, __builtin_convertvector((f32x2{a - back[0], b - back[1]}), tx2));
}

// A score in the exp2 domain: LOG2E (softcap tanh(s scale / softcap) + bias); bias in the exp2 domain, with the cap's constant
// folded in:  softcap tanh(u) = softcap - 2 softcap / (e^(2u) + 1)
struct ScoreScale { float a, b, c0; };
__device__ __forceinline__ ScoreScale score_scale(const GqaCall& c) {
  if (c.softcap > 0.f) return ScoreScale{2.0f * LOG2E * c.scale / c.softcap, -2.0f * c.softcap * LOG2E, c.softcap * LOG2E};
  return ScoreScale{c.scale * LOG2E, 0.f, 0.f};
}
template <bool CAP>
__device__ __forceinline__ float score2(const ScoreScale& k, float s, float bias) {
  if constexpr (CAP) return fmaf(k.b, __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(s * k.a) + 1.0f), bias);
  else return fmaf(s, k.a, bias);
}

// 1 / (1 + e^-z) on the hardware's exponential and reciprocal (a last bit each)
__device__ __forceinline__ float gate_f(float z) { return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-LOG2E * z)); }

// How many keys back the distance bias leaves anything: a capped score is at most softcap and the token's own at least -softcap, so
// a key further away than this has a weight below 2^-40 of the token's own -- nothing in a float32 sum
__device__ __forceinline__ int key_reach(const GqaCall& c, float slope2) {
  if (c.softcap <= 0.f || slope2 <= 0.f) return 1 << 30;
  return (int)fminf((2.0f * LOG2E * c.softcap + 40.0f) / slope2, 1e9f) + 1;
}

// The same for a block whose scores all stay below 0.6 softcap / scale: softcap tanh(s scale / softcap) = s P(s^2), P a polynomial
// (least-squares fit of tanh(u) / u at Chebyshev points, |u| <= 0.6: relative error 1.6e-7) -- no transcendentals
struct CapPoly { float c[5], lim; };
__device__ __forceinline__ CapPoly cap_poly(const GqaCall& c) {
  const float f = c.scale / c.softcap, f2 = f * f;
  CapPoly k;
  k.c[0] = c.scale * LOG2E;
  k.c[1] = -0.33332324028015137f * f2 * k.c[0];
  k.c[2] = 0.13310357928276062f * f2 * f2 * k.c[0];
  k.c[3] = -0.052109625190496445f * f2 * f2 * f2 * k.c[0];
  k.c[4] = 0.01548669021576643f * f2 * f2 * f2 * f2 * k.c[0];
  k.lim = 0.6f / fabsf(f);
  return k;
}
__device__ __forceinline__ float score_poly(const CapPoly& k, float s, float bias) {
  const float w = s * s;
  return fmaf(s, fmaf(fmaf(fmaf(fmaf(k.c[4], w, k.c[3]), w, k.c[2]), w, k.c[1]), w, k.c[0]), bias);
}

// N consecutive elements, n of them there (the rest zero): one load where N divides n
template <typename T, int N>
__device__ __forceinline__ void load_upto(const T* p, int k, int n, float (&v)[N]) {
  typedef T tv __attribute__((ext_vector_type(N)));
  if (n % N == 0 && ((uintptr_t)p & (N * sizeof(T) - 1)) == 0) {
    const tv x = *(const tv*)(p + min(k, n - N));
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] = k < n ? to_f32(x[i]) : 0.f;
  } else {
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] = k + i < n ? to_f32(p[k + i]) : 0.f;
  }
}

// grid (nsplit, G x head tiles, nd), 4 waves; a wave walks its 32-key blocks on its own, the next block's loads in flight during
// the current one.  The token's own key and value are added by the last split from LDS, which also appends them (shared: they are in
// the cache already).
template <typename T, int KD, int VD, bool PAGED, bool CAP>
__global__ __launch_bounds__(256, 1) void gqa_decode_kernel(GqaCall c) {
  constexpr int KK = KD / 32, DT = VD / 16, KB = 32, IMG = KB * VD * 2, NV = KB * VD / 8 / 64, LQ = KD + 8;
  static_assert(IMG == 16 * VD * 4, "a wave's value image holds its 16 output rows");
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];      // 4 value images; later [5][16][VD] outputs
  __shared__ __attribute__((aligned(16))) T qs[16 * LQ];
  __shared__ __attribute__((aligned(16))) T kn[KD];
  __shared__ float vn[VD];
  __shared__ float st_m[5 * 16], st_l[5 * 16];
  __shared__ int last_sh;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c16 = lane & 15, g4 = lane >> 4;
  const int rep = c.H / c.G, ht_n = (rep + 15) / 16;
  const int split = blockIdx.x, kh = blockIdx.y / ht_n, ht = blockIdx.y % ht_n, m = blockIdx.z;
  const int seg = c.t.dec[m], row = c.t.row[seg], tok = c.t.tok0[seg], pos = c.t.off[row];
  const int h0 = kh * rep + ht * 16, nh = min(16, rep - ht * 16);
  const int end = pos + (c.shared ? 1 : 0);
  const int lo = max(first_seen(c, pos), pos - key_reach(c, c.slopes[h0 + nh - 1] * LOG2E));     // cached keys [lo, end) (the slopes fall)
  const int kept = min(c.keep, pos);                                                             // and [0, kept)
  const int blk0 = lo / KB, nmain = end > lo ? (end + KB - 1) / KB - blk0 : 0;
  const int nkept = nmain > 0 ? min((kept + KB - 1) / KB, blk0) : (kept + KB - 1) / KB, nblk = nkept + nmain;
  const int per = (nblk + c.nsplit - 1) / c.nsplit, b0 = split * per, b1 = min(b0 + per, nblk);
  auto block_of = [&](int i) { return i < nkept ? i : blk0 + i - nkept; };
  const T* kc = (const T*)c.kcache;
  const T* vc = (const T*)c.vcache;
  unsigned char* img = smem + wave * IMG;
  u32x4 kf[2][KK], vr[NV];
  auto load_k = [&](int blk) {
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      const T* p = kc + kv_elem<PAGED>(c.sk, row, kh, max(0, min(blk * KB + 16 * t + c16, end - 1))) + 8 * g4;
#pragma unroll
      for (int kk = 0; kk < KK; ++kk) kf[t][kk] = *(const u32x4*)(p + 32 * kk);
    }
  };
  auto load_v = [&](int blk) {
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int piece = i * 64 + lane;
      vr[i] = *(const u32x4*)(vc + kv_elem<PAGED>(c.sv, row, kh, max(0, min(blk * KB + piece / (VD / 8), end - 1))) + 8 * (piece % (VD / 8)));
    }
  };

  // queries (and, in the last split, the token's own key and value): 16 lanes per head.  Their loads go first: memory answers in order
  const T* pr = (const T*)c.proj + (size_t)tok * c.ldp;
  const bool own = split == c.nsplit - 1 && !c.shared;
  {
    const int hh = tid >> 4, l = tid & 15;
    constexpr int PL = KD / 16;                      // elements per lane: l PL ..
    float vq[PL], wq[PL], vk[PL], wk[PL];
    Rot<PL> rq, rk;
    const bool key_lanes = own && tid < 16;
    load_upto<T, PL>(pr + c.o_q + (h0 + min(hh, nh - 1)) * c.dim, l * PL, c.dim, vq);
    load_upto<float, PL>(c.q_norm, l * PL, c.dim, wq);
    if (key_lanes) {
      load_upto<T, PL>(pr + c.o_k + kh * c.dim, l * PL, c.dim, vk);
      load_upto<float, PL>(c.k_norm, l * PL, c.dim, wk);
    }
    if (c.rot > 0) {
      load_rot<T, PL>(c, pr + c.o_q + (h0 + min(hh, nh - 1)) * c.dim, c.q_norm, l * PL, pos, rq);
      if (key_lanes) load_rot<T, PL>(c, pr + c.o_k + kh * c.dim, c.k_norm, l * PL, pos, rk);
    }
    if (b0 + wave < b1) { load_k(block_of(b0 + wave)); load_v(block_of(b0 + wave)); }
    auto head = [&](const float (&v)[PL], const float (&w)[PL], const Rot<PL>& ro, bool there, T* dst) {
      float ss = 0.f, x[PL];
#pragma unroll
      for (int i = 0; i < PL; ++i) ss += v[i] * v[i] * square_weight(c, l * PL + i);
      const float rs = 1.0f / sqrtf(row16_sum(ss) / (float)c.dim + c.eps);
#pragma unroll
      for (int i = 0; i < PL; ++i) x[i] = v[i] * rs * w[i];
      if (c.rot > 0) rotate<PL>(ro, rs, x);
#pragma unroll
      for (int i = 0; i < PL; ++i) dst[l * PL + i] = from_f32<T>(there ? x[i] : 0.f);
    };
    head(vq, wq, rq, hh < nh, qs + hh * LQ);
    if (key_lanes) head(vk, wk, rk, true, kn);
    if (own && tid >= 64 && tid < 64 + VD) {
      const int k = tid - 64;
      float x = 0.f;
      if (k < c.vdim) {
        x = to_f32(pr[c.o_v + kh * c.vdim + k]);
        const size_t fo = (size_t)tok * c.G * c.vdim + kh * c.vdim + k;
        if (c.v_first_out != nullptr && ht == 0) ((T*)c.v_first_out)[fo] = from_f32<T>(x);
        if (c.v_mix != nullptr) { const float lam = *c.v_mix; x = (1.0f - lam) * x + lam * to_f32(((const T*)c.v_first_in)[fo]); }
      }
      const T xt = from_f32<T>(x);
      vn[k] = to_f32(xt);
      if (ht == 0) ((T*)c.vcache)[kv_elem<PAGED>(c.sv, row, kh, pos) + k] = xt;
    }
  }
  __syncthreads();
  if (own && ht == 0 && tid < KD) ((T*)c.kcache)[kv_elem<PAGED>(c.sk, row, kh, pos) + tid] = kn[tid];
  u32x4 qf[KK];
#pragma unroll
  for (int kk = 0; kk < KK; ++kk) qf[kk] = *(const u32x4*)(qs + c16 * LQ + 32 * kk + 8 * g4);
  const ScoreScale ks = score_scale(c);
  const float slope2 = c.slopes[h0 + min(c16, nh - 1)] * LOG2E;
  float m_run = -1e30f, l_run = 0.f;
  f32x4 acc[DT];
#pragma unroll
  for (int dt = 0; dt < DT; ++dt) acc[dt] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int tq4 = c16 >> 2, tp = c16 & 3;

  for (int it = b0 + wave; it < b1; it += 4) {
    const int blk = block_of(it);
    f32x4 sc[2];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      sc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < KK; ++kk) sc[t] = mfma16<T>(kf[t][kk], qf[kk], sc[t]);
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int piece = i * 64 + lane, key = piece / (VD / 8), dc = piece % (VD / 8);
      *(u32x4*)(img + (size_t)(dc >> 1) * (KB * 32) + key * 32 + (dc & 1) * 16) = vr[i];
    }
    if (it + 4 < b1) { load_k(block_of(it + 4)); load_v(block_of(it + 4)); }
    float mx = -INFINITY;
    const float bias0 = fmaf(slope2, (float)(blk * KB + 4 * g4 - pos), ks.c0);
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = blk * KB + 16 * t + 4 * g4 + r;
        const float s = score2<CAP>(ks, sc[t][r], fmaf(slope2, (float)(16 * t + r), bias0));
        sc[t][r] = (key >= lo && key < end) || key < kept ? s : -INFINITY;
        mx = fmaxf(mx, sc[t][r]);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float mn = fmaxf(m_run, mx);
    if (__builtin_amdgcn_ballot_w64(mn != m_run) != 0) {
      const float corr = __builtin_amdgcn_exp2f(m_run - mn);
      m_run = mn;
      l_run *= corr;
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) acc[dt] *= corr;
    }
    uint32_t ph[4], pw[4];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      float p[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) { p[r] = __builtin_amdgcn_exp2f(sc[t][r] - mn); l_run += p[r]; }
      split2<T>(p[0], p[1], ph[2 * t], pw[2 * t]);
      split2<T>(p[2], p[3], ph[2 * t + 1], pw[2 * t + 1]);
    }
    const u32x4 pf = {ph[0], ph[1], ph[2], ph[3]}, pl = {pw[0], pw[1], pw[2], pw[3]};
    asm volatile("" ::: "memory");                   // (a wave's LDS operations complete in order)
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      const unsigned char* a0 = img + (size_t)dt * (KB * 32) + (4 * g4 + tq4) * 32 + tp * 8;
      const s16x4 v0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)a0);
      const s16x4 v1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)(a0 + 16 * 32));
      const uint32_t* w0 = (const uint32_t*)&v0;
      const uint32_t* w1 = (const uint32_t*)&v1;
      const u32x4 vf = {w0[0], w0[1], w1[0], w1[1]};
      acc[dt] = mfma16<T>(vf, pf, acc[dt]);
      acc[dt] = mfma16<T>(vf, pl, acc[dt]);
    }
    asm volatile("" ::: "memory");
    __builtin_amdgcn_wave_barrier();
  }
  l_run += __shfl_xor(l_run, 16, 64);
  l_run += __shfl_xor(l_run, 32, 64);
  // this wave's maximum, weight sum and outputs of the heads in columns c16 (its own image is free)
  float* of = (float*)smem;                          // [5][16][VD]
#pragma unroll
  for (int dt = 0; dt < DT; ++dt) *(f32x4*)(of + (size_t)(wave * 16 + c16) * VD + 16 * dt + 4 * g4) = acc[dt];
  if (g4 == 0) { st_m[wave * 16 + c16] = m_run; st_l[wave * 16 + c16] = l_run; }
  {                                                  // entry 4: the token's own key and value
    const int hh = tid >> 4, l = tid & 15;
    float s = 0.f;
    if (own) {
#pragma unroll
      for (int i = 0; i < KD / 16; ++i) s = fmaf(to_f32(qs[hh * LQ + l * (KD / 16) + i]), to_f32(kn[l * (KD / 16) + i]), s);
    }
    s = row16_sum(s);
    if (l == 0) { st_m[64 + hh] = own ? score2<CAP>(ks, s, ks.c0) : -1e30f; st_l[64 + hh] = own ? 1.0f : 0.f; }
    for (int i = tid; i < 16 * VD; i += 256) of[64 * VD + i] = own ? vn[i % VD] : 0.f;
  }
  __syncthreads();
  T* cat = (T*)c.cat + (size_t)tok * c.ldc;
  const bool gated = c.o_g >= 0;
  const T* gate = pr + max(c.o_g, 0);
  auto sink_of = [&](int h, float mn) { return c.sink != nullptr ? __builtin_amdgcn_exp2f(c.sink[h] * LOG2E - mn) : 0.f; };
  float* pp0 = c.partial + (size_t)m * c.H * c.nsplit * (VD + 2);
  for (int idx = tid; idx < nh * VD; idx += 256) {
    const int hh = idx / VD, d = idx % VD;
    float mn = -1e30f;
#pragma unroll
    for (int w = 0; w < 5; ++w) mn = fmaxf(mn, st_m[w * 16 + hh]);
    float L = 0.f, O = 0.f;
#pragma unroll
    for (int w = 0; w < 5; ++w) {
      const float cw = __builtin_amdgcn_exp2f(st_m[w * 16 + hh] - mn);
      L = fmaf(st_l[w * 16 + hh], cw, L);
      O = fmaf(of[(size_t)(w * 16 + hh) * VD + d], cw, O);
    }
    const int h = h0 + hh;
    if (c.nsplit == 1) {
      L += sink_of(h, mn);
      if (d < c.vdim) cat[h * c.vdim + d] = from_f32<T>(gated ? O / L * gate_f(to_f32(gate[gate_at(c, h, d)])) : O / L);
    } else {
      float* pp = pp0 + ((size_t)h * c.nsplit + split) * (VD + 2);
      __hip_atomic_store(&pp[2 + d], O, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
      if (d == 0) {
        __hip_atomic_store(&pp[0], mn, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        __hip_atomic_store(&pp[1], L, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
      }
    }
  }
  if (c.nsplit == 1) return;
  // the last split to arrive combines (nobody waits): partials are at agent scope, the ticket follows them
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();
  if (tid == 0) {
    int* ctr = &c.counters[m * gridDim.y + blockIdx.y];
    const int ticket = __hip_atomic_fetch_add(ctr, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    last_sh = ticket == c.nsplit - 1;
    if (last_sh) __hip_atomic_store(ctr, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  }
  __syncthreads();
  if (!last_sh) return;
  for (int idx = tid; idx < nh * VD; idx += 256) {
    const int hh = idx / VD, d = idx % VD, h = h0 + hh;
    const float* pp = pp0 + (size_t)h * c.nsplit * (VD + 2);
    const float gv = gated ? to_f32(gate[gate_at(c, h, min(d, c.vdim - 1))]) : 0.f;
    float mn = -1e30f, L = 0.f, O = 0.f;
    for (int i0 = 0; i0 < c.nsplit; i0 += 8) {       // eight splits' loads in flight, merged in split order
      float mv[8], lv[8], ov[8];
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float* q = pp + (size_t)min(i0 + j, c.nsplit - 1) * (VD + 2);
        mv[j] = __hip_atomic_load(&q[0], __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        lv[j] = __hip_atomic_load(&q[1], __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        ov[j] = __hip_atomic_load(&q[2 + d], __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
      }
      float bm = mn;
#pragma unroll
      for (int j = 0; j < 8; ++j) if (i0 + j < c.nsplit) bm = fmaxf(bm, mv[j]);
      const float cs = __builtin_amdgcn_exp2f(mn - bm);
      L *= cs; O *= cs; mn = bm;
#pragma unroll
      for (int j = 0; j < 8; ++j)
        if (i0 + j < c.nsplit) {
          const float cw = __builtin_amdgcn_exp2f(mv[j] - bm);
          L = fmaf(lv[j], cw, L);
          O = fmaf(ov[j], cw, O);
        }
    }
    L += sink_of(h, mn);
    if (d < c.vdim) cat[h * c.vdim + d] = from_f32<T>(gated ? O / L * gate_f(gv) : O / L);
  }
}

// grid (H, query tiles), 4 waves of 16 QG queries each; all waves share the head's keys and values: blocks of 64 keys from the
// tile's last one downwards (then the kept tokens' blocks), two LDS buffers, the next block's global loads in flight during the current block's MFMAs.
// Downwards because of the distance bias: the running maximum is found in the first block and seldom moves.  It lags: a block's
// weights are taken relative to the maximum of the blocks before it, and only a score more than 8 (a factor 256) above that makes
// the wave find the new maximum and rescale -- no cross-lane step in most blocks.
// LDS images, XOR-ed so that the 16-byte writes of consecutive lanes hit different banks:
//   K [16-key tile][kk][g][key ^ (4 kk + g)] x 16 B     V [32 keys][16-value tile dt][key ^ (dt & 7)] x 32 B
// PG: 0 contiguous cache, 1 pages of 64 tokens and more (one page per block of keys), 2 smaller pages
template <typename T, int KD, int VD, int QG, int PG, bool CAP>
__global__ __launch_bounds__(256, 2) void gqa_prefill_kernel(GqaCall c) {
  constexpr int KB = 64, KK = KD / 32, DT = VD / 16, KT = KB / 16, KIMG = KB * KD * 2, VIMG = KB * VD * 2;
  constexpr int NKP = KB * KD / 8 / 256, NVP = KB * VD / 8 / 256;      // 16-byte pieces per thread
  constexpr float UNSET = -1e30f, LAG = 8.0f;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];  // K[2], V[2]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c16 = lane & 15, g4 = lane >> 4;
  const int seg = c.t.tile[2 * blockIdx.y], t0 = c.t.tile[2 * blockIdx.y + 1], h = blockIdx.x, kh = h / (c.H / c.G);
  const int row = c.t.row[seg], len = c.t.len[seg], off = c.t.off[row], tok0 = c.t.tok0[seg];
  const float slope2 = c.slopes[h] * LOG2E;
  const int nk = off + min(t0 + 64 * QG, len);       // keys any query of the tile may see: [first, nk)
  const int first = max(first_seen(c, off + t0), off + t0 - key_reach(c, slope2));
  const int jlast = (nk - 1) / KB, jfirst = first / KB, nmain = jlast - jfirst + 1;
  const int nkept = min((c.keep + KB - 1) / KB, jfirst), nblk = nmain + nkept;                   // blocks in front of jfirst that hold kept tokens
  auto block_of = [&](int i) { i = min(i, nblk - 1); return i < nmain ? jlast - i : nblk - 1 - i; };
  const T* kc = (const T*)c.kcache;
  const T* vc = (const T*)c.vcache;
  auto kimg = [&](int b) { return smem + b * KIMG; };
  auto vimg = [&](int b) { return smem + 2 * KIMG + b * VIMG; };

  // key block j of the cache: element of its first key (PG 0, 1); `page` is looked up one block ahead of its use
  const int32_t* btab = PG ? c.sk.btab + (size_t)row * c.sk.bt_stride : nullptr;
  int page = 0;
  auto find_page = [&](int j) { if constexpr (PG == 1) page = __builtin_amdgcn_readfirstlane(btab[(j * KB) >> c.sk.bs_shift]); };
  auto block_at = [&](const AttnShape& s, int j) -> size_t {
    if constexpr (PG == 0) return (((size_t)row * s.Hkv + kh) * s.cap + (size_t)j * KB) * s.D;
    else return ((((size_t)page * s.Hkv + kh) << s.bs_shift) + (size_t)((j * KB) & ((1 << s.bs_shift) - 1))) * s.D;
  };
  u32x4 kreg[NKP], vreg[NVP];
  auto load_block = [&](int j) {                     // (keys beyond nk are read as the last one: the cache may end there)
    const int top = min(nk - 1 - j * KB, KB - 1);
    if constexpr (PG == 2) {
#pragma unroll
      for (int i = 0; i < NKP; ++i) {
        const int piece = i * 256 + tid;
        kreg[i] = *(const u32x4*)(kc + kv_elem<true>(c.sk, row, kh, j * KB + min(piece / (KD / 8), top)) + 8 * (piece % (KD / 8)));
      }
#pragma unroll
      for (int i = 0; i < NVP; ++i) {
        const int piece = i * 256 + tid;
        vreg[i] = *(const u32x4*)(vc + kv_elem<true>(c.sv, row, kh, j * KB + min(piece / (VD / 8), top)) + 8 * (piece % (VD / 8)));
      }
    } else {
      const T* kb = kc + block_at(c.sk, j);
      const T* vb = vc + block_at(c.sv, j);
#pragma unroll
      for (int i = 0; i < NKP; ++i) {
        const int piece = i * 256 + tid, key = min(piece / (KD / 8), top);
        kreg[i] = *(const u32x4*)(kb + key * KD + 8 * (piece % (KD / 8)));
      }
#pragma unroll
      for (int i = 0; i < NVP; ++i) {
        const int piece = i * 256 + tid, key = min(piece / (VD / 8), top);
        vreg[i] = *(const u32x4*)(vb + key * VD + 8 * (piece % (VD / 8)));
      }
    }
  };
  auto store_block = [&](int buf) {
#pragma unroll
    for (int i = 0; i < NKP; ++i) {
      const int piece = i * 256 + tid, key = piece / (KD / 8), dc = piece % (KD / 8);
      *(u32x4*)(kimg(buf) + (((key >> 4) * KK * 4 + dc) * 16 + ((key ^ dc) & 15)) * 16) = kreg[i];
    }
#pragma unroll
    for (int i = 0; i < NVP; ++i) {
      const int piece = i * 256 + tid, key = piece / (VD / 8), dc = piece % (VD / 8);
      *(u32x4*)(vimg(buf) + (size_t)((key >> 5) * DT + (dc >> 1)) * (32 * 32) + ((key & 31) ^ ((dc >> 1) & 7)) * 32 + (dc & 1) * 16) = vreg[i];
    }
  };
  find_page(jlast);
  load_block(jlast);
  find_page(block_of(1));
  u32x4 qf[QG][KK];
  int tq[QG], lo[QG];                                // this lane's query of group u and the first key of its chunk or window
#pragma unroll
  for (int u = 0; u < QG; ++u) {
    tq[u] = t0 + (wave * QG + u) * 16 + c16;
    lo[u] = first_seen(c, off + tq[u]);
    const T* q = (const T*)c.q + ((size_t)(tok0 + min(tq[u], len - 1)) * c.H + h) * KD;
#pragma unroll
    for (int kk = 0; kk < KK; ++kk) qf[u][kk] = *(const u32x4*)(q + 32 * kk + 8 * g4);
  }
  store_block(0);
#pragma unroll
  for (int u = 0; u < QG; ++u)
#pragma unroll
    for (int kk = 0; kk < KK; ++kk) asm volatile("" :: "v"(qf[u][kk]));      // (loaded from here on: no wait carried round the loop)
  __syncthreads();
  const ScoreScale ks = score_scale(c);
  CapPoly kp{};
  if constexpr (CAP) kp = cap_poly(c);
  float m_run[QG], l_run[QG];
  f32x4 acc[QG][DT];
#pragma unroll
  for (int u = 0; u < QG; ++u) {
    m_run[u] = UNSET; l_run[u] = 0.f;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) acc[u][dt] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const int tq4 = c16 >> 2, tp = c16 & 3;
  for (int it = 0; it < nblk; ++it) {
    const int j = block_of(it), buf = it & 1;
    load_block(block_of(it + 1));                 // straight-line (behind the last block: that block again, not stored): a
    find_page(block_of(it + 2));                         // conditional load would make the compiler wait for all loads at the loop's head
    f32x4 sc[QG][KT];
#pragma unroll
    for (int t = 0; t < KT; ++t) {
#pragma unroll
      for (int u = 0; u < QG; ++u) sc[u][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < KK; ++kk) {
        const u32x4 kf = *(const u32x4*)(kimg(buf) + (((t * KK + kk) * 4 + g4) * 16 + (c16 ^ ((4 * kk + g4) & 15))) * 16);
#pragma unroll
        for (int u = 0; u < QG; ++u) sc[u][t] = mfma16<T>(kf, qf[u][kk], sc[u][t]);
      }
    }
    u32x4 pf[QG][2], pl[QG][2];
#pragma unroll
    for (int u = 0; u < QG; ++u) {
      const int q0 = off + t0 + (wave * QG + u) * 16;    // position of the group's first query
      // scores relative to the running maximum
      const float ref = m_run[u] == UNSET ? 0.f : m_run[u];
      const float bias0 = fmaf(slope2, (float)(j * KB + 4 * g4 - (q0 + c16)), -ref);
      bool small = CAP;
      if constexpr (CAP) {
        float am = 0.f;
#pragma unroll
        for (int t = 0; t < KT; ++t)
#pragma unroll
          for (int r = 0; r < 4; ++r) am = fmaxf(am, fabsf(sc[u][t][r]));
        small = __builtin_amdgcn_ballot_w64(am > kp.lim) == 0;
      }
      if (small) {
#pragma unroll
        for (int t = 0; t < KT; ++t)
#pragma unroll
          for (int r = 0; r < 4; ++r) sc[u][t][r] = score_poly(kp, sc[u][t][r], fmaf(slope2, (float)(16 * t + r), bias0));
      } else {
#pragma unroll
        for (int t = 0; t < KT; ++t)
#pragma unroll
          for (int r = 0; r < 4; ++r) sc[u][t][r] = score2<CAP>(ks, sc[u][t][r], fmaf(slope2, (float)(16 * t + r), bias0 + ks.c0));
      }
      // a block that reaches past the first query, or in front of the last query's chunk or window (uniform)
      if (j * KB + KB - 1 > q0 || j * KB < first_seen(c, q0 + 15)) {
#pragma unroll
        for (int t = 0; t < KT; ++t)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int key = j * KB + 16 * t + 4 * g4 + r;
            sc[u][t][r] = key <= q0 + c16 && (key >= lo[u] || key < c.keep) ? sc[u][t][r] : -INFINITY;
          }
      }
      float mx = -INFINITY;
#pragma unroll
      for (int t = 0; t < KT; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) mx = fmaxf(mx, sc[u][t][r]);
      if (__builtin_amdgcn_ballot_w64(mx > LAG || m_run[u] == UNSET) != 0) {
        mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        const float mn = fmaxf(m_run[u], ref + mx);                    // (UNSET while the query has seen no key)
        const float corr = __builtin_amdgcn_exp2f(m_run[u] - mn), d = (mn == UNSET ? 0.f : mn) - ref;
        m_run[u] = mn;
        l_run[u] *= corr;
#pragma unroll
        for (int dt = 0; dt < DT; ++dt) acc[u][dt] *= corr;
#pragma unroll
        for (int t = 0; t < KT; ++t)
#pragma unroll
          for (int r = 0; r < 4; ++r) sc[u][t][r] -= d;
      }
#pragma unroll
      for (int hf = 0; hf < 2; ++hf) {
        uint32_t ph[4], pw[4];
#pragma unroll
        for (int t = 0; t < 2; ++t) {
          float p[4];
#pragma unroll
          for (int r = 0; r < 4; ++r) { p[r] = __builtin_amdgcn_exp2f(sc[u][2 * hf + t][r]); l_run[u] += p[r]; }
          split2<T>(p[0], p[1], ph[2 * t], pw[2 * t]);
          split2<T>(p[2], p[3], ph[2 * t + 1], pw[2 * t + 1]);
        }
        pf[u][hf] = u32x4{ph[0], ph[1], ph[2], ph[3]};
        pl[u][hf] = u32x4{pw[0], pw[1], pw[2], pw[3]};
      }
    }
#pragma unroll
    for (int hf = 0; hf < 2; ++hf)
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) {
        const unsigned char* a0 = vimg(buf) + (size_t)(hf * DT + dt) * (32 * 32) + ((4 * g4 + tq4) ^ (dt & 7)) * 32 + tp * 8;
        const s16x4 v0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)a0);
        const s16x4 v1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)(a0 + 16 * 32));
        const uint32_t* w0 = (const uint32_t*)&v0;
        const uint32_t* w1 = (const uint32_t*)&v1;
        const u32x4 vf = {w0[0], w0[1], w1[0], w1[1]};
#pragma unroll
        for (int u = 0; u < QG; ++u) acc[u][dt] = mfma16<T>(vf, pf[u][hf], acc[u][dt]);
#pragma unroll
        for (int u = 0; u < QG; ++u) acc[u][dt] = mfma16<T>(vf, pl[u][hf], acc[u][dt]);
      }
    if (it + 1 < nblk) store_block(buf ^ 1);             // the other buffer: nobody reads it during this block
    __syncthreads();
  }
  // output: the gates of a query are fetched in one round trip
#pragma unroll
  for (int u = 0; u < QG; ++u) {
    float l = l_run[u];
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (c.sink != nullptr) l += __builtin_amdgcn_exp2f(c.sink[h] * LOG2E - m_run[u]);
    const int tok = tok0 + min(tq[u], len - 1);
    const bool gated = c.o_g >= 0 && !c.gate_head;
    const T* gates = (const T*)c.proj + (size_t)tok * c.ldp + max(c.o_g, 0);
    const T* gate = gates + (c.gate_head ? 0 : h * c.vdim);
    const float inv = (c.o_g >= 0 && c.gate_head ? gate_f(to_f32(gates[h])) : 1.0f) / l;
    T* o = (T*)c.cat + (size_t)tok * c.ldc + h * c.vdim;
    if (c.vdim % 4 == 0) {
      uint2 gt[DT];
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) gt[dt] = gated ? *(const uint2*)(gate + min(16 * dt + 4 * g4, c.vdim - 4)) : uint2{0, 0};
      if (tq[u] >= len) continue;
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) {
        const int k = 16 * dt + 4 * g4;
        const T* ge = (const T*)&gt[dt];
        T v[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = (T)(acc[u][dt][r] * inv * (gated ? gate_f(to_f32(ge[r])) : 1.0f));
        if (k < c.vdim) *(uint2*)(o + k) = __builtin_bit_cast(uint2, v);
      }
    } else if (tq[u] < len) {
#pragma unroll
      for (int dt = 0; dt < DT; ++dt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int k = 16 * dt + 4 * g4 + r;
          if (k < c.vdim) o[k] = (T)(acc[u][dt][r] * inv * (gated ? gate_f(to_f32(gate[k])) : 1.0f));
        }
    }
  }
}

template <typename T>
int pre_at(const GqaCall& c, hipStream_t st) {
  const bool vec = c.dim % 8 == 0 && c.vdim % 8 == 0 && c.kdp <= 128 && c.vdp <= 128 && (c.pairs || c.rot % 16 == 0);
  auto go = [&](auto k) { hipLaunchKernelGGL(k, dim3(c.t.R), dim3(256), 0, st, c); };
  if (c.rot > 0) { if (vec) go(gqa_pre_kernel<T, true, true>); else go(gqa_pre_kernel<T, false, true>); }
  else { if (vec) go(gqa_pre_kernel<T, true, false>); else go(gqa_pre_kernel<T, false, false>); }
  MI_HIP(hipGetLastError());
  return MI_OK;
}

template <typename T>
int generic_at(const GqaCall& c, hipStream_t st) {
  const dim3 grid(c.t.R, c.H), block(256);
  const size_t lds = (size_t)4 * c.vdp * sizeof(float);
  const int nr = (std::max(c.dim, c.vdim) + 63) / 64;
#define GO(N) hipLaunchKernelGGL((gqa_generic_kernel<T, N>), grid, block, lds, st, c)
  if (nr <= 1) GO(1); else if (nr <= 2) GO(2); else if (nr <= 4) GO(4); else if (nr <= 8) GO(8);
  else return fail(MI_ERR_UNSUPPORTED, "gqa: head sizes above 512");
#undef GO
  MI_HIP(hipGetLastError());
  return MI_OK;
}

template <typename T, int KD, int VD>
int decode_kv(const GqaCall& c, hipStream_t st) {
  constexpr int lds = 5 * 16 * VD * 4;
  const dim3 grid(c.nsplit, c.G * gqa_head_tiles(c.H, c.G), c.t.nd);
  auto go = [&](auto kern) -> int {
    hipLaunchKernelGGL(kern, grid, dim3(256), lds, st, c);
    MI_HIP(hipGetLastError());
    return MI_OK;
  };
  if (c.softcap > 0.f) return c.sk.btab ? go(gqa_decode_kernel<T, KD, VD, true, true>) : go(gqa_decode_kernel<T, KD, VD, false, true>);
  return c.sk.btab ? go(gqa_decode_kernel<T, KD, VD, true, false>) : go(gqa_decode_kernel<T, KD, VD, false, false>);
}

template <typename T, int KD, int VD>
int prefill_kv(const GqaCall& c, hipStream_t st) {
  constexpr int lds = 2 * 64 * (KD + VD) * 2;
  auto go = [&](auto kern) -> int {
    MI_HIP(hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, lds));
    hipLaunchKernelGGL(kern, dim3(c.H, c.t.nt), dim3(256), lds, st, c);
    MI_HIP(hipGetLastError());
    return MI_OK;
  };
  const int pg = c.sk.btab == nullptr ? 0 : (c.sk.bs_shift >= 6 ? 1 : 2);
#define GO(CAP) (pg == 0 ? go(gqa_prefill_kernel<T, KD, VD, 1, 0, CAP>) : (pg == 1 ? go(gqa_prefill_kernel<T, KD, VD, 1, 1, CAP>) : go(gqa_prefill_kernel<T, KD, VD, 1, 2, CAP>)))
  return c.softcap > 0.f ? GO(true) : GO(false);
#undef GO
}

template <typename T, bool DECODE>
int fast_at(const GqaCall& c, hipStream_t st) {
#define V(KD, VD) if (c.kdp == KD && c.vdp == VD) { if constexpr (DECODE) return decode_kv<T, KD, VD>(c, st); else return prefill_kv<T, KD, VD>(c, st); }
  V(32, 32) V(32, 64) V(32, 128) V(64, 32) V(64, 64) V(64, 128) V(128, 32) V(128, 64) V(128, 128)
#undef V
  return fail(MI_ERR_UNSUPPORTED, "gqa: head sizes");
}

#define BY_ACT(fn) \
  switch (c.act) { \
    case MI_F32: return fn<float>(c, st); \
    case MI_BF16: return fn<bf16>(c, st); \
    case MI_F16: return fn<f16>(c, st); \
  } \
  return fail(MI_ERR_INVALID, "gqa: bad dtype")

int check_call(const GqaCall& c) {
  if (c.G < 1 || c.H % c.G != 0 || c.sk.D != c.kdp || c.sv.D != c.vdp || c.sk.Hkv != c.G || c.sv.Hkv != c.G || c.kdp < c.dim || c.vdp < c.vdim)
    return fail(MI_ERR_INVALID, "gqa: cache shape does not match the layer");
  if (c.rot < 0 || c.rot % 2 != 0 || c.rot > c.dim || (c.rot > 0 && c.rot_tab == nullptr)) return fail(MI_ERR_INVALID, "gqa: rotation does not fit the head size");
  if (c.shared && (c.v_mix != nullptr || c.v_first_out != nullptr)) return fail(MI_ERR_INVALID, "gqa: mixed values need a layer's own");
  if (c.window < 0 || c.keep < 0 || (c.window > 0 && c.chunk > 0) || (c.window == 0 && c.keep > 0)) return fail(MI_ERR_INVALID, "gqa: bad mask");
  return MI_OK;
}

}  // namespace

int gqa_pad(int n) { return n <= 32 ? 32 : (n <= 64 ? 64 : (n <= 128 ? 128 : (n + 31) / 32 * 32)); }
bool gqa_supported(int dim, int vdim) { return dim >= 1 && vdim >= 1 && dim <= 512 && vdim <= 512; }
bool gqa_mfma_supported(int act, int dim, int vdim) { return (act == MI_BF16 || act == MI_F16) && dim <= 128 && vdim <= 128; }

int launch_gqa_pre(const GqaCall& c, hipStream_t st) { MI_TRY(check_call(c)); BY_ACT(pre_at); }
int launch_gqa_generic(const GqaCall& c, hipStream_t st) { MI_TRY(check_call(c)); BY_ACT(generic_at); }
int launch_gqa_decode(const GqaCall& c, hipStream_t st) {
  MI_TRY(check_call(c));
  if (c.nsplit < 1 || (c.nsplit > 1 && (c.partial == nullptr || c.counters == nullptr))) return fail(MI_ERR_INVALID, "gqa_decode: bad split configuration");
  if (c.act == MI_BF16) return fast_at<bf16, true>(c, st);
  if (c.act == MI_F16) return fast_at<f16, true>(c, st);
  return fail(MI_ERR_UNSUPPORTED, "gqa_decode: 16-bit caches only");
}
int launch_gqa_prefill(const GqaCall& c, hipStream_t st) {
  MI_TRY(check_call(c));
  if (c.t.qt != 64) return fail(MI_ERR_INVALID, "gqa_prefill: tiles of 64 queries");
  if (c.act == MI_BF16) return fast_at<bf16, false>(c, st);
  if (c.act == MI_F16) return fast_at<f16, false>(c, st);
  return fail(MI_ERR_UNSUPPORTED, "gqa_prefill: 16-bit caches only");
}

}  // namespace mi
