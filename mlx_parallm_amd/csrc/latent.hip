// latent.hip -- latent attention (layer-list models): the cache holds one latent c per token, head h's keys and values are W_uk c and
// W_uv c, scores (q . k) * scale, ordinary causal softmax, the head's output times sigmoid(gate) (or no gate).
// With a rotated part every query head has `rot` more coordinates, turned by the position; the keys' are one vector per token for all
// heads, turned and cached behind the latent.  A score is then ([W_uk^T q | q_rot] . [c | k_rot]) * scale: the latent space has more
// coordinates, which only the scores look at.  Where keys are materialised, [W_uk | 1] hands the rotated part through.
//
//   generic form     any size and dtype: the query goes into the latent space (W_uk^T q), scores and the weighted sum are taken
//                    over the latents, W_uv is applied to the sum.  One workgroup per (token, head), float32 arithmetic.
//   latent_decode    16-bit caches, one-token segments: the same absorption on the matrix cores; the heads of a token share
//                    every latent that is read (16 heads = the columns of one MFMA).
//   latent_prefill   16-bit caches, longer segments: keys and values are materialised once per call (one GEMM over the gathered
//                    latents), then flash attention with tiles of 64 queries.
#include <algorithm>
#include <type_traits>

#include "layer_rows.h"

namespace mi {

namespace {

using namespace rows;

template <bool PAGED>
__device__ __forceinline__ size_t lat_elem(const AttnShape& s, int row, int key) { return kv_elem<PAGED>(s, row, 0, key); }
__device__ __forceinline__ size_t lat_at(const AttnShape& s, int row, int key) {
  return s.btab ? kv_elem<true>(s, row, 0, key) : kv_elem<false>(s, row, 0, key);
}

// coordinate j of a rotated part at position pos, x: the part as projected
template <typename T>
__device__ __forceinline__ float rotated(const LatentCall& c, const T* x, int j, int pos) {
  const RotAt a = rot_at(j, c.rot, c.pairs);
  const float2 cs = c.rot_tab[(size_t)pos * (c.rot >> 1) + a.f];
  return to_f32(x[j]) * cs.x + a.sign * to_f32(x[a.partner]) * cs.y;
}

// grid (rows / RPW, parts): c = rms(W_dkv h) * w and the rotated key part appended to the cache; the feed-forward activation of the row;
// the latent of the queries.  A wave takes a row of a norm; the feed-forward needs the whole workgroup (RPW = 1: the norms' other
// waves are idle).
enum : int { PRE_CACHE, PRE_FF, PRE_QUERY };
inline int pre_parts(const LatentCall& c) { return (c.o_c >= 0 ? 1 : 0) + (c.ff.ff > 0 ? 1 : 0) + (c.q_rank > 0 ? 1 : 0); }
__device__ __forceinline__ int pre_part(const LatentCall& c, int i) {
  if (c.o_c >= 0 && i-- == 0) return PRE_CACHE;
  if (c.ff.ff > 0 && i-- == 0) return PRE_FF;
  return PRE_QUERY;
}
template <typename T, int RPW>
__global__ __launch_bounds__(256) void latent_pre_kernel(LatentCall c) {
  __shared__ float red[12];
  const int part = pre_part(c, blockIdx.y), lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  if constexpr (RPW == 1) {
    if (part == PRE_FF) {
      const int r = blockIdx.x;
      polynorm_row<T, 256>(c.ff, (const T*)c.proj + (size_t)r * c.ldp + c.ff.in_off, (T*)c.cat + (size_t)r * c.ldc + c.ff.out_off, red);
      return;
    }
  }
  const int r = __builtin_amdgcn_readfirstlane(blockIdx.x * RPW + wave);
  if (wave >= RPW || r >= c.t.R) return;
  const bool cache = part == PRE_CACHE;
  const int n = cache ? c.rank : c.q_rank, np = cache ? c.rp : c.ldqc;
  const T* src = (const T*)c.proj + (size_t)r * c.ldp + (cache ? c.o_c : c.o_qc);       // (parts of a projected row begin at multiples of 16)
  const float* w = cache ? c.c_norm : c.q_norm;
  const TokenAt at = token_at(c.t, r);
  T* dst = cache ? (T*)c.cache + lat_at(c.s, at.row, at.pos) : (T*)c.qc + (size_t)r * c.ldqc;
  // pieces of eight: [0, n) the norm's, [cp, cp + rot) the rotated key part, zeros between and behind (cp is a multiple of 16)
  auto in_rot = [&](int k) { return cache && k >= c.cp && k < c.cp + c.rot; };
  auto load = [&](int k, float (&x)[8], float (&g)[8]) {
    if (k + 8 <= n) {
      load8f<T>(src + k, x);
      load8f<float>(w + k, g);
      return;
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      x[i] = g[i] = 0.f;
      if (k + i < n) { x[i] = to_f32(src[k + i]); g[i] = w[k + i]; }
      else if (in_rot(k) && k + i < c.cp + c.rot) g[i] = rotated<T>(c, src + n, k + i - c.cp, at.pos);       // (x = 0: not the norm's)
    }
  };
  constexpr int KEEP = 2;                              // pieces per lane that stay in registers
  float x[KEEP][8], g[KEEP][8], ss = 0.f;
#pragma unroll
  for (int p = 0; p < KEEP; ++p) load(8 * (lane + 64 * p), x[p], g[p]);
#pragma unroll
  for (int p = 0; p < KEEP; ++p)
#pragma unroll
    for (int i = 0; i < 8; ++i) ss += x[p][i] * x[p][i];
  for (int k = 8 * (lane + 64 * KEEP); k < n; k += 512) {
    float y[8], z[8];
    load(k, y, z);
#pragma unroll
    for (int i = 0; i < 8; ++i) ss += y[i] * y[i];
  }
  const float rs = 1.0f / sqrtf(wave_sum(ss) / (float)n + c.eps);
  auto put = [&](int k, float (&y)[8], const float (&z)[8]) {
    if (k >= np) return;
    const bool rot = in_rot(k);
#pragma unroll
    for (int i = 0; i < 8; ++i) y[i] = rot ? z[i] : y[i] * rs * z[i];
    store8f<T>(dst + k, y);
  };
#pragma unroll
  for (int p = 0; p < KEEP; ++p) put(8 * (lane + 64 * p), x[p], g[p]);
  for (int k = 8 * (lane + 64 * KEEP); k < np; k += 512) {
    float y[8], z[8];
    load(k, y, z);
    put(k, y, z);
  }
}

// gate of token r and head h
template <typename T>
__device__ __forceinline__ float head_gate(const LatentCall& c, int r, int h) {
  return c.o_g >= 0 ? sigmoid_f(to_f32(((const T*)c.proj)[(size_t)r * c.ldp + c.o_g + h])) : 1.f;
}

// ---- generic form --------------------------------------------------------------------------------------------------
// grid (R, H): lq[r][h][:] = [W_uk^T q | rotated part]
template <typename T>
__global__ __launch_bounds__(256) void latent_absorb_generic_kernel(LatentCall c) {
  const int r = blockIdx.x, h = blockIdx.y;
  const T* q = (const T*)c.q + (size_t)r * c.ldq + h * (c.dim + c.rot);
  const T* uk = (const T*)c.uk + (size_t)h * c.dim * c.rank;
  const int pos = c.rot > 0 ? token_at(c.t, r).pos : 0;
  float* out = (float*)c.lq + ((size_t)r * c.H + h) * c.rp;
  for (int k = threadIdx.x; k < c.rp; k += 256) {
    float a = 0.f;
    if (k < c.rank)
      for (int j = 0; j < c.dim; ++j) a = fmaf(to_f32(q[j]), to_f32(uk[(size_t)j * c.rank + k]), a);
    else if (k >= c.cp && k < c.cp + c.rot) a = rotated<T>(c, q + c.dim, k - c.cp, pos);
    out[k] = a;
  }
}

// grid (R, H), 4 waves: wave w takes keys w, w + 4, ..; NR latent elements per lane
template <typename T, int NR>
__global__ __launch_bounds__(256) void latent_attn_generic_kernel(LatentCall c) {
  extern __shared__ float sm[];                      // [4][rp] sums, then [rp] merged
  __shared__ float ml[8];
  const int r = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const TokenAt at = token_at(c.t, r);
  const float* lq = (const float*)c.lq + ((size_t)r * c.H + h) * c.rp;
  const T* cache = (const T*)c.cache;
  float q[NR], o[NR], m = -INFINITY, l = 0.f;
#pragma unroll
  for (int i = 0; i < NR; ++i) { const int k = lane + 64 * i; q[i] = k < c.rp ? lq[k] * c.scale : 0.f; o[i] = 0.f; }
  constexpr int U = NR <= 4 ? 4 : 2;                 // keys in flight
  for (int key = wave; key <= at.pos; key += 4 * U) {
    float x[U][NR], sc[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const T* p = cache + lat_at(c.s, at.row, min(key + 4 * u, at.pos));
#pragma unroll
      for (int i = 0; i < NR; ++i) { const int k = lane + 64 * i; x[u][i] = k < c.rp ? to_f32(p[k]) : 0.f; }
    }
    float mx = m;
#pragma unroll
    for (int u = 0; u < U; ++u) {
      float a = 0.f;
#pragma unroll
      for (int i = 0; i < NR; ++i) a = fmaf(q[i], x[u][i], a);
      sc[u] = wave_sum(a);
      if (key + 4 * u <= at.pos) mx = fmaxf(mx, sc[u]);
    }
    const float corr = expf(m - mx);                 // (the first key of the loop is visible: mx is finite)
    m = mx; l *= corr;
#pragma unroll
    for (int i = 0; i < NR; ++i) o[i] *= corr;
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const float p = key + 4 * u <= at.pos ? expf(sc[u] - m) : 0.f;
      l += p;
#pragma unroll
      for (int i = 0; i < NR; ++i) o[i] = fmaf(p, x[u][i], o[i]);
    }
  }
#pragma unroll
  for (int i = 0; i < NR; ++i) { const int k = lane + 64 * i; if (k < c.rp) sm[wave * c.rp + k] = o[i]; }
  if (lane == 0) { ml[wave] = m; ml[4 + wave] = l; }
  __syncthreads();
  const float mx = fmaxf(fmaxf(ml[0], ml[1]), fmaxf(ml[2], ml[3]));
  float w[4], lt = 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) { w[i] = expf(ml[i] - mx); lt += w[i] * ml[4 + i]; }
  for (int k = threadIdx.x; k < c.rp; k += 256)
    sm[k] = (w[0] * sm[k] + w[1] * sm[c.rp + k] + w[2] * sm[2 * c.rp + k] + w[3] * sm[3 * c.rp + k]) / lt;
  __syncthreads();
  const float gate = head_gate<T>(c, r, h);
  const T* uv = (const T*)c.uv + (size_t)h * c.vdim * c.rank;
  T* cat = (T*)c.cat + (size_t)r * c.ldc + h * c.vdim;
  for (int j = wave; j < c.vdim; j += 4) {
    float a = 0.f;
    for (int k = lane; k < c.rank; k += 64) a = fmaf(sm[k], to_f32(uv[(size_t)j * c.rank + k]), a);
    a = wave_sum(a);
    if (lane == 0) cat[j] = from_f32<T>(a * gate);
  }
}

template <typename T>
int generic_at(const LatentCall& c, hipStream_t st) {
  hipLaunchKernelGGL(latent_absorb_generic_kernel<T>, dim3(c.t.R, c.H), dim3(256), 0, st, c);
  MI_HIP(hipGetLastError());
  const dim3 grid(c.t.R, c.H), block(256);
  const size_t lds = (size_t)4 * c.rp * sizeof(float);
  const int nr = (c.rp + 63) / 64;
#define GO(N) hipLaunchKernelGGL((latent_attn_generic_kernel<T, N>), grid, block, lds, st, c)
  if (nr <= 1) GO(1); else if (nr <= 2) GO(2); else if (nr <= 4) GO(4); else if (nr <= 8) GO(8); else if (nr <= 16) GO(16);
  else return fail(MI_ERR_UNSUPPORTED, "latent attention: kv_rank above 1024");
#undef GO
  MI_HIP(hipGetLastError());
  return MI_OK;
}

}  // namespace

#define BY_ACT(fn) \
  switch (c.act) { \
    case MI_F32: return fn<float>(c, st); \
    case MI_BF16: return fn<bf16>(c, st); \
    case MI_F16: return fn<f16>(c, st); \
  } \
  return fail(MI_ERR_INVALID, "latent attention: bad dtype")

template <typename T>
static int pre_at(const LatentCall& c, hipStream_t st) {
  const int parts = pre_parts(c);
  if (parts == 0) return MI_OK;
  if (c.ff.ff > 0) hipLaunchKernelGGL((latent_pre_kernel<T, 1>), dim3(c.t.R, parts), dim3(256), 0, st, c);
  else hipLaunchKernelGGL((latent_pre_kernel<T, 4>), dim3((c.t.R + 3) / 4, parts), dim3(256), 0, st, c);
  MI_HIP(hipGetLastError());
  return MI_OK;
}
int launch_latent_pre(const LatentCall& c, hipStream_t st) { BY_ACT(pre_at); }
int launch_latent_generic(const LatentCall& c, hipStream_t st) { BY_ACT(generic_at); }

// ---- matrix-core forms ----------------------------------------------------------------------------------------------
namespace {

typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef _Float16 f16x8 __attribute__((ext_vector_type(8)));
constexpr float LOG2E = 1.4426950408889634f;
constexpr int LAT_PART_PAD = 4;      // a split's partial row: rp sums, running maximum, weight sum (padded to 16 bytes)

template <typename T>
__device__ __forceinline__ f32x4 mfma16(u32x4 a, u32x4 b, f32x4 c) {
  if constexpr (std::is_same<T, bf16>::value)
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
  else
    return __builtin_amdgcn_mfma_f32_16x16x32_f16(__builtin_bit_cast(f16x8, a), __builtin_bit_cast(f16x8, b), c, 0, 0, 0);
}

// two float32 values as hi + lo pairs of 16-bit values (float32 weights / queries as two exact-ish MFMA operands)
template <typename T>
__device__ __forceinline__ void split2(float a, float b, uint32_t& hi, uint32_t& lo) {
  typedef float f32x2 __attribute__((ext_vector_type(2)));
  typedef T tx2 __attribute__((ext_vector_type(2)));
  const tx2 h = __builtin_convertvector((f32x2{a, b}), tx2);
  const f32x2 back = __builtin_convertvector(h, f32x2);
  hi = __builtin_bit_cast(uint32_t, h);
  lo = __builtin_bit_cast(uint32_t, __builtin_convertvector((f32x2{a - back[0], b - back[1]}), tx2));
}

// elements [k, k + 8) of a vector of n, zeros beyond n
template <typename T>
__device__ __forceinline__ u32x4 load8_upto(const T* p, int k, int n) {
  if (n % 8 == 0 && ((uintptr_t)p & 15) == 0) {
    if (k < n) return *(const u32x4*)(p + k);
    return u32x4{0, 0, 0, 0};
  }
  T v[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) v[i] = k + i < n ? p[k + i] : (T)0.f;
  return __builtin_bit_cast(u32x4, v);
}

// elements [k, k + 8) of query head qh [dim | rot] with the rotated part turned, zeros beyond
template <typename T>
__device__ __forceinline__ u32x4 query8(const LatentCall& c, const T* qh, int k, int pos) {
  const u32x4 x = load8_upto<T>(qh, k, c.dim + c.rot);
  if (c.rot == 0 || k + 8 <= c.dim || k >= c.dim + c.rot) return x;
  T v[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const int j = k + i - c.dim;
    v[i] = ((const T*)&x)[i];
    if (j >= 0 && j < c.rot) v[i] = from_f32<T>(rotated<T>(c, qh + c.dim, j, pos));
  }
  return __builtin_bit_cast(u32x4, v);
}

// one-token segments: lq[m][h] = [W_uk^T q | rotated part] as a 16-bit pair hi + lo.  grid (H, rp / 64, ceil(nd / 16)); a wave owns 16
// columns (cp is a multiple of 16)
template <typename T>
__global__ __launch_bounds__(256) void latent_absorb_kernel(LatentCall c) {
  const int h = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c16 = lane & 15, g4 = lane >> 4;
  const int r0 = blockIdx.y * 64 + wave * 16, m0 = blockIdx.z * 16;
  const int m = min(m0 + c16, c.t.nd - 1);
  const T* q = (const T*)c.q + (size_t)c.t.tok0[c.t.dec[m]] * c.ldq + h * (c.dim + c.rot);
  const T* w = (const T*)c.uk_t + ((size_t)h * c.rp + r0 + c16) * c.kdp;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  if (c.rot > 0 && r0 >= c.cp) {
    const int j = r0 + c16 - c.cp;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int seg = c.t.dec[min(m0 + 4 * g4 + r, c.t.nd - 1)];
      if (j < c.rot) acc[r] = rotated<T>(c, (const T*)c.q + (size_t)c.t.tok0[seg] * c.ldq + h * (c.dim + c.rot) + c.dim, j, c.t.off[c.t.row[seg]]);
    }
  } else for (int k = 0; k < c.dim; k += 32)           // (kdp is a multiple of 32 and at least dim)
    acc = mfma16<T>(load8_upto<T>(q, k + 8 * g4, c.dim), *(const u32x4*)(w + k + 8 * g4), acc);
  T* out = (T*)c.lq;                                 // [m][h][hi | lo][rp]
#pragma unroll
  for (int r = 0; r < 4; ++r)
    if (m0 + 4 * g4 + r < c.t.nd) {
      T* o = out + ((size_t)(m0 + 4 * g4 + r) * c.H + h) * 2 * c.rp + r0 + c16;
      const T hi = (T)acc[r];
      o[0] = hi;
      o[c.rp] = (T)(acc[r] - (float)hi);
    }
}

// grid (nsplit, head tiles, nd), 4 waves; a wave walks its 32-key blocks on its own (no barrier in the loop).
//   S^T = C Q^T: A = latents straight from global memory (row = key), B = queries (column = head), hi + lo
//   O^T = C^T P: the same registers go to a wave-private LDS image [16-element tile][key][16 elements], read back transposed
template <typename T, int NK, bool PAGED>
__global__ __launch_bounds__(256, 1) void latent_decode_kernel(LatentCall c) {
  constexpr int RP = 64 * NK, KK = RP / 32, DT = RP / 16, KB = 32, IMG = KB * RP * 2;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  __shared__ float ml[2][4][16];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c16 = lane & 15, g4 = lane >> 4;
  const int m = blockIdx.z, ht = blockIdx.y, seg = c.t.dec[m], row = c.t.row[seg];
  const int n = c.t.off[row] + 1;                    // visible keys
  const int nblk = (n + KB - 1) / KB, per = (nblk + c.nsplit - 1) / c.nsplit;
  const int b0 = blockIdx.x * per, b1 = min(b0 + per, nblk);
  unsigned char* img = smem + wave * IMG;
  const T* cache = (const T*)c.cache;

  u32x4 qh[KK], ql[KK];
  {
    const int head = min(ht * 16 + c16, c.H - 1);
    const T* q = (const T*)c.lq + ((size_t)m * c.H + head) * 2 * RP + 8 * g4;
#pragma unroll
    for (int kk = 0; kk < KK; ++kk) { qh[kk] = *(const u32x4*)(q + 32 * kk); ql[kk] = *(const u32x4*)(q + RP + 32 * kk); }
  }
  const float sc2 = c.scale * LOG2E;
  float m_run = -1e30f, l_run = 0.f;
  f32x4 acc[DT];
#pragma unroll
  for (int dt = 0; dt < DT; ++dt) acc[dt] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int tq4 = c16 >> 2, tp = c16 & 3;

  for (int blk = b0 + wave; blk < b1; blk += 4) {
    u32x4 kf[2][KK];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      const T* p = cache + lat_elem<PAGED>(c.s, row, min(blk * KB + 16 * t + c16, n - 1)) + 8 * g4;
#pragma unroll
      for (int kk = 0; kk < KK; ++kk) kf[t][kk] = *(const u32x4*)(p + 32 * kk);
    }
    f32x4 sc[2];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      sc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < KK; ++kk) {
        sc[t] = mfma16<T>(kf[t][kk], qh[kk], sc[t]);
        sc[t] = mfma16<T>(kf[t][kk], ql[kk], sc[t]);
      }
    }
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int kk = 0; kk < KK; ++kk)
        *(u32x4*)(img + (size_t)(2 * kk + (g4 >> 1)) * (KB * 32) + (16 * t + c16) * 32 + (g4 & 1) * 16) = kf[t][kk];
    float mx = -INFINITY;
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        sc[t][r] = blk * KB + 16 * t + 4 * g4 + r < n ? sc[t][r] : -INFINITY;
        mx = fmaxf(mx, sc[t][r]);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float mn = fmaxf(m_run, mx * sc2);         // (scale > 0)
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
      for (int r = 0; r < 4; ++r) { p[r] = __builtin_amdgcn_exp2f(fmaf(sc[t][r], sc2, -mn)); l_run += p[r]; }
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
  // merge the four waves: O^T lies as [head][rp] floats in the wave's own image
  float* of = (float*)img;
#pragma unroll
  for (int dt = 0; dt < DT; ++dt) *(f32x4*)(of + (size_t)c16 * RP + 16 * dt + 4 * g4) = acc[dt];
  if (g4 == 0) { ml[0][wave][c16] = m_run; ml[1][wave][c16] = l_run; }
  __syncthreads();
  const int nh = min(16, c.H - ht * 16);
  const int ht_n = (c.H + 15) / 16;
  for (int hh = wave; hh < nh; hh += 4) {
    const float mx = fmaxf(fmaxf(ml[0][0][hh], ml[0][1][hh]), fmaxf(ml[0][2][hh], ml[0][3][hh]));
    float w[4], lt = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) { w[i] = __builtin_amdgcn_exp2f(ml[0][i][hh] - mx); lt += w[i] * ml[1][i][hh]; }
    float* dst = c.partial + (((size_t)m * ht_n * 16 + ht * 16 + hh) * c.nsplit + blockIdx.x) * (RP + LAT_PART_PAD);
    for (int k = lane; k < RP; k += 64) {
      float a = 0.f;
#pragma unroll
      for (int i = 0; i < 4; ++i) a += w[i] * ((const float*)(smem + i * IMG))[(size_t)hh * RP + k];
      dst[k] = a;
    }
    if (lane == 0) { dst[RP] = mx; dst[RP + 1] = lt; }
  }
}

// merge the splits: c.merged[m][h] = the weighted sum of the latents as a 16-bit pair hi + lo.  grid (H, nd), four latent elements per thread (rp <= 768)
template <typename T>
__global__ __launch_bounds__(192) void latent_merge_kernel(LatentCall c) {
  const int h = blockIdx.x, m = blockIdx.y, ns = c.nsplit, lp = c.rp + LAT_PART_PAD, lane = threadIdx.x & 63, k = threadIdx.x * 4;
  const float* p = c.partial + ((size_t)m * ((c.H + 15) / 16 * 16) + h) * ns * lp;
  // lane s holds the weight of split s (at most 32 of them)
  const float* e = p + (size_t)min(lane, ns - 1) * lp + c.rp;
  const float mv = e[0], lv = e[1];
  float mx = mv;
#pragma unroll
  for (int x = 1; x < 64; x *= 2) mx = fmaxf(mx, __shfl_xor(mx, x, 64));
  float w = lane < ns ? __builtin_amdgcn_exp2f(mv - mx) : 0.f;
  w /= wave_sum(w * lv);
  f32x4 a = {0.f, 0.f, 0.f, 0.f};
  for (int s = 0; s < ns; s += 8) {
    f32x4 v[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = *(const f32x4*)(p + (size_t)min(s + j, ns - 1) * lp + min(k, c.rp - 4));
#pragma unroll
    for (int j = 0; j < 8; ++j) a += v[j] * __shfl(w, s + j, 64);        // (zero beyond the last split)
  }
  if (k >= c.rp) return;
  uint32_t hi[2], lo[2];
  split2<T>(a[0], a[1], hi[0], lo[0]);
  split2<T>(a[2], a[3], hi[1], lo[1]);
  T* dst = (T*)c.merged + ((size_t)m * c.H + h) * 2 * c.rp + k;
  *(uint2*)dst = uint2{hi[0], hi[1]};
  *(uint2*)(dst + c.rp) = uint2{lo[0], lo[1]};
}

// W_uv and the gate.  grid (ceil(vdim / 16), H, ceil(nd / 16)), one wave of 16 tokens and 16 output columns
template <typename T, int NK>
__global__ __launch_bounds__(64) void latent_uv_kernel(LatentCall c) {
  const int lane = threadIdx.x, c16 = lane & 15, g4 = lane >> 4;
  const int h = blockIdx.y, m0 = blockIdx.z * 16, nm = min(16, c.t.nd - m0);
  const int col = blockIdx.x * 16 + c16;
  const T* w = (const T*)c.uv_p + ((size_t)h * c.vdim + min(col, c.vdim - 1)) * c.rp + 8 * g4;
  const T* x = (const T*)c.merged + ((size_t)(m0 + min(c16, nm - 1)) * c.H + h) * 2 * c.rp + 8 * g4;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f}, acc1 = {0.f, 0.f, 0.f, 0.f};
  u32x4 b[2 * NK], xh[2 * NK], xl[2 * NK];            // (all loads in one round trip)
#pragma unroll
  for (int k = 0; k < 2 * NK; ++k) {
    b[k] = *(const u32x4*)(w + 32 * k);
    xh[k] = *(const u32x4*)(x + 32 * k);
    xl[k] = *(const u32x4*)(x + c.rp + 32 * k);
  }
  __builtin_amdgcn_sched_barrier(0);
#pragma unroll
  for (int k = 0; k < 2 * NK; ++k) {
    acc = mfma16<T>(xh[k], b[k], acc);
    acc1 = mfma16<T>(xl[k], b[k], acc1);
  }
  acc += acc1;
  if (col >= c.vdim) return;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int m = 4 * g4 + r;
    if (m >= nm) continue;
    const int tok = c.t.tok0[c.t.dec[m0 + m]];
    const float gate = head_gate<T>(c, tok, h);
    ((T*)c.cat)[(size_t)tok * c.ldc + h * c.vdim + col] = from_f32<T>(acc[r] * gate);
  }
}

// grid key tiles: the latents a chunk attends to (cached and new), contiguous
template <typename T>
__global__ __launch_bounds__(256) void latent_gather_kernel(LatentCall c, T* dst) {
  const int seg = c.t.gtile[2 * blockIdx.x], k0 = c.t.gtile[2 * blockIdx.x + 1], row = c.t.row[seg];
  const int n = min(LATENT_GT, c.t.off[row] + c.t.len[seg] - k0), np = c.rp / 8;
  for (int i = threadIdx.x; i < n * np; i += 256) {
    const int key = i / np, pc = i % np;
    *(u32x4*)(dst + (size_t)(c.t.kbase[seg] + k0 + key) * c.rp + 8 * pc) =
        *(const u32x4*)((const T*)c.cache + lat_at(c.s, row, k0 + key) + 8 * pc);
  }
}

// grid (query tiles, H), 4 waves of 16 QG queries each; all waves share the head's keys and values: blocks of 64 keys from the
// diagonal downwards, two LDS buffers, the next block's global loads in flight during the current block's MFMAs.  The running maximum
// lags: weights are taken relative to that of the blocks before, and only a score more than 8 (a factor 256) above it makes the wave
// find the new one and rescale -- no cross-lane step in most blocks.
// LDS images, XOR-ed so that the 16-byte writes of consecutive lanes hit different banks:
//   K [16-key tile][piece of eight][key ^ piece] x 16 B     V [32 keys][16-value tile dt][key ^ (dt & 7)] x 32 B
template <typename T, int KD, int VD, int QG>
__global__ __launch_bounds__(256, 2) void latent_prefill_kernel(LatentCall c) {
  constexpr int KB = 64, KK = KD / 32, DT = VD / 16, KT = KB / 16, KIMG = KB * KD * 2, VIMG = KB * VD * 2;
  constexpr int NKP = KB * KD / 8 / 256, NVP = KB * VD / 8 / 256;      // 16-byte pieces per thread
  constexpr float UNSET = -1e30f, LAG = 8.0f;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];  // K[2], V[2]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c16 = lane & 15, g4 = lane >> 4;
  const int seg = c.t.tile[2 * blockIdx.x], t0 = c.t.tile[2 * blockIdx.x + 1], h = blockIdx.y;
  const int row = c.t.row[seg], len = c.t.len[seg], off = c.t.off[row], tok0 = c.t.tok0[seg];
  const int nk = off + min(t0 + 64 * QG, len);       // keys any query of the tile may see
  const int nb = (nk + KB - 1) / KB;
  const T* kp = (const T*)c.kv + (size_t)c.t.kbase[seg] * c.ldkv + h * KD;
  const T* vp = (const T*)c.kv + (size_t)c.t.kbase[seg] * c.ldkv + c.H * KD + h * VD;
  auto kimg = [&](int b) { return smem + b * KIMG; };
  auto vimg = [&](int b) { return smem + 2 * KIMG + b * VIMG; };

  u32x4 kreg[NKP], vreg[NVP];
  auto load_block = [&](int j) {                     // (keys beyond nk are read as the last one)
    const T* kb = kp + (size_t)j * KB * c.ldkv;
    const T* vb = vp + (size_t)j * KB * c.ldkv;
    const int top = min(nk - 1 - j * KB, KB - 1);
#pragma unroll
    for (int i = 0; i < NKP; ++i) {
      const int piece = i * 256 + tid;
      kreg[i] = *(const u32x4*)(kb + (uint32_t)min(piece / (KD / 8), top) * (uint32_t)c.ldkv + 8 * (piece % (KD / 8)));
    }
#pragma unroll
    for (int i = 0; i < NVP; ++i) {
      const int piece = i * 256 + tid;
      vreg[i] = *(const u32x4*)(vb + (uint32_t)min(piece / (VD / 8), top) * (uint32_t)c.ldkv + 8 * (piece % (VD / 8)));
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
  load_block(nb - 1);
  u32x4 qf[QG][KK];
  int tq[QG];
#pragma unroll
  for (int u = 0; u < QG; ++u) {
    tq[u] = t0 + (wave * QG + u) * 16 + c16;
    const int tc = min(tq[u], len - 1);
    const T* q = (const T*)c.q + (size_t)(tok0 + tc) * c.ldq + h * (c.dim + c.rot);
#pragma unroll
    for (int kk = 0; kk < KK; ++kk) qf[u][kk] = query8<T>(c, q, 32 * kk + 8 * g4, off + tc);
  }
  store_block(0);
#pragma unroll
  for (int u = 0; u < QG; ++u)
#pragma unroll
    for (int kk = 0; kk < KK; ++kk) asm volatile("" :: "v"(qf[u][kk]));      // (loaded from here on: no wait carried round the loop)
  __syncthreads();
  const float sc2 = c.scale * LOG2E;                   // (positive)
  float m_run[QG], l_run[QG];
  f32x4 acc[QG][DT];
#pragma unroll
  for (int u = 0; u < QG; ++u) {
    m_run[u] = UNSET; l_run[u] = 0.f;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) acc[u][dt] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const int tq4 = c16 >> 2, tp = c16 & 3;
  for (int it = 0; it < nb; ++it) {
    const int j = nb - 1 - it, buf = it & 1;
    load_block(max(j - 1, 0));                         // straight-line (behind the last block: that one again, not stored)
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
      const float ref = m_run[u] == UNSET ? 0.f : m_run[u];
#pragma unroll
      for (int t = 0; t < KT; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) sc[u][t][r] = fmaf(sc[u][t][r], sc2, -ref);          // relative to the running maximum
      if (j * KB + KB - 1 > q0) {                        // a block that reaches past it (uniform)
#pragma unroll
        for (int t = 0; t < KT; ++t)
#pragma unroll
          for (int r = 0; r < 4; ++r) sc[u][t][r] = j * KB + 16 * t + 4 * g4 + r <= q0 + c16 ? sc[u][t][r] : -INFINITY;
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
    if (it + 1 < nb) store_block(buf ^ 1);               // the other buffer: nobody reads it during this block
    __syncthreads();
  }
#pragma unroll
  for (int u = 0; u < QG; ++u) {
    float l = l_run[u];
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (tq[u] >= len) continue;
    const int tok = tok0 + tq[u];
    const float f = head_gate<T>(c, tok, h) / l;
    T* o = (T*)c.cat + (size_t)tok * c.ldc + h * c.vdim;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      const int k = 16 * dt + 4 * g4;
      if (c.vdim % 4 == 0) {
        if (k < c.vdim) {
          T v[4] = {(T)(acc[u][dt][0] * f), (T)(acc[u][dt][1] * f), (T)(acc[u][dt][2] * f), (T)(acc[u][dt][3] * f)};
          *(uint2*)(o + k) = __builtin_bit_cast(uint2, v);
        }
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r) if (k + r < c.vdim) o[k + r] = (T)(acc[u][dt][r] * f);
      }
    }
  }
}

template <typename T, int NK>
int decode_nk(const LatentCall& c, hipStream_t st) {
  const dim3 grid(c.nsplit, (c.H + 15) / 16, c.t.nd), block(256);
  const int lds = 4 * 32 * 64 * NK * 2;
  auto go = [&](auto kern) -> int {
    MI_HIP(hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, lds));
    hipLaunchKernelGGL(kern, grid, block, lds, st, c);
    MI_HIP(hipGetLastError());
    return MI_OK;
  };
  if (c.s.btab) MI_TRY(go(latent_decode_kernel<T, NK, true>));
  else MI_TRY(go(latent_decode_kernel<T, NK, false>));
  hipLaunchKernelGGL(latent_merge_kernel<T>, dim3(c.H, c.t.nd), dim3(c.rp <= 512 ? 128 : 192), 0, st, c);
  MI_HIP(hipGetLastError());
  hipLaunchKernelGGL((latent_uv_kernel<T, NK>), dim3((c.vdim + 15) / 16, c.H, (c.t.nd + 15) / 16), dim3(64), 0, st, c);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

template <typename T>
int decode_at(const LatentCall& c, hipStream_t st) {
  if constexpr (sizeof(T) == 2) {
    hipLaunchKernelGGL(latent_absorb_kernel<T>, dim3(c.H, c.rp / 64, (c.t.nd + 15) / 16), dim3(256), 0, st, c);
    MI_HIP(hipGetLastError());
    switch (c.rp / 64) {
      case 1: return decode_nk<T, 1>(c, st);
      case 2: return decode_nk<T, 2>(c, st);
      case 3: return decode_nk<T, 3>(c, st);
      case 4: return decode_nk<T, 4>(c, st);
      case 5: return decode_nk<T, 5>(c, st);
      case 6: return decode_nk<T, 6>(c, st);
      case 7: return decode_nk<T, 7>(c, st);
      case 8: return decode_nk<T, 8>(c, st);
      case 9: return decode_nk<T, 9>(c, st);
    }
    return fail(MI_ERR_UNSUPPORTED, "latent_decode: latent size");
  } else return fail(MI_ERR_UNSUPPORTED, "latent_decode: 16-bit caches only");
}

template <typename T, int KD, int VD>
int prefill_kv(const LatentCall& c, hipStream_t st) {
  const int lds = 2 * 64 * (KD + VD) * 2;
  auto go = [&](auto kern) -> int {
    MI_HIP(hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, lds));
    hipLaunchKernelGGL(kern, dim3(c.t.nt, c.H), dim3(256), lds, st, c);
    MI_HIP(hipGetLastError());
    return MI_OK;
  };
  if constexpr (KD + VD < 256) {                       // (larger heads do not fit the registers)
    if (c.t.qt == 128) return go(latent_prefill_kernel<T, KD, VD, 2>);
  }
  if (c.t.qt != 64) return fail(MI_ERR_INVALID, "latent_prefill: tile size");
  return go(latent_prefill_kernel<T, KD, VD, 1>);
}

template <typename T>
int prefill_at(const LatentCall& c, hipStream_t st) {
  if constexpr (sizeof(T) == 2) {
#define V(KD) switch (c.vdp) { case 32: return prefill_kv<T, KD, 32>(c, st); case 64: return prefill_kv<T, KD, 64>(c, st); case 128: return prefill_kv<T, KD, 128>(c, st); } break
    switch (c.kdp) {
      case 32: V(32);
      case 64: V(64);
      case 128: V(128);
      case 192: V(192);
    }
#undef V
  }
  return fail(MI_ERR_UNSUPPORTED, "latent_prefill: head sizes / dtype");
}

template <typename T>
int gather_at(const LatentCall& c, void* dst, hipStream_t st) {
  if constexpr (sizeof(T) == 2) {
    hipLaunchKernelGGL(latent_gather_kernel<T>, dim3(c.t.ngt), dim3(256), 0, st, c, (T*)dst);
    MI_HIP(hipGetLastError());
    return MI_OK;
  } else return fail(MI_ERR_UNSUPPORTED, "latent_gather: 16-bit caches only");
}

}  // namespace

int latent_pad(int n) { return n <= 32 ? 32 : (n <= 64 ? 64 : (n <= 128 ? 128 : 0)); }
int latent_tile(int kdp, int vdp) { return kdp + vdp < 256 ? 128 : 64; }
int latent_key_pad(int n) { return n > 128 && n <= 192 ? 192 : latent_pad(n); }
bool latent_mfma_supported(int act, int dim, int vdim, int rp) {
  return (act == MI_BF16 || act == MI_F16) && latent_key_pad(dim) > 0 && latent_pad(vdim) > 0 && rp % 64 == 0 && rp <= 576;
}
int launch_latent_decode(const LatentCall& c, hipStream_t st) {
  if (c.nsplit < 1 || c.nsplit > 32 || c.partial == nullptr) return fail(MI_ERR_INVALID, "latent_decode: bad split configuration");
  BY_ACT(decode_at);
}
int launch_latent_gather(const LatentCall& c, void* dst, hipStream_t st) {
  switch (c.act) {
    case MI_BF16: return gather_at<bf16>(c, dst, st);
    case MI_F16: return gather_at<f16>(c, dst, st);
  }
  return fail(MI_ERR_UNSUPPORTED, "latent_gather: 16-bit caches only");
}
int launch_latent_prefill(const LatentCall& c, hipStream_t st) { BY_ACT(prefill_at); }

}  // namespace mi
