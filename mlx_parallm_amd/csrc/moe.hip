// moe.hip -- mixture of experts (layer-list models): a softmax router picks `top` experts per token among the `keep` best of
// `groups` equal groups; an expert is W_down glu(W_gate h, W_up h) (common.h: Glu); the shared expert takes all tokens.  The weighted sum
// over a token's slots is taken by the row kernel behind (layer_rows.hip: post_norm_kernel).
//
//   route       many rows: router logits on the matrix cores (x as hi + lo, so they keep 32-bit accuracy, or h), softmax, groups, choice
//               (few rows and float32: inside post_norm_kernel)
//   plan        many rows: slots sorted by expert, table of tiles, for the grouped tile GEMM (gemm_prefill.hip)
//   stream      up to MOE_STREAM_ROWS tokens: one workgroup per (expert, strip of weight rows) collects the expert's slots and
//               streams its weights once per 16 or 32 of them
//   generic     any dtype, row-major weights: one workgroup per (slot, strip of rows), float32 arithmetic
#include <algorithm>
#include <type_traits>

#include "layer_rows.h"

namespace mi {

namespace {

using namespace rows;

typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef _Float16 f16x8 __attribute__((ext_vector_type(8)));

template <typename T>
__device__ __forceinline__ f32x4 mfma16(u32x4 a, u32x4 b, f32x4 c) {
  if constexpr (std::is_same<T, bf16>::value)
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
  else
    return __builtin_amdgcn_mfma_f32_16x16x32_f16(__builtin_bit_cast(f16x8, a), __builtin_bit_cast(f16x8, b), c, 0, 0, 0);
}

// ---- router of many rows: 16 rows per workgroup, RTW waves split K ---------------------------------------------------------
template <typename T, int NE, int RTW, bool H16>       // NE: 16-expert tiles; H16: the rows are h
__global__ __launch_bounds__(RTW * 64) void route_kernel(MoeCall c) {
  extern __shared__ __attribute__((aligned(16))) float sm[];      // partial tiles [RTW][NE][64][4]; then logits [16][16 NE], per wave weights | marks, choices
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c16 = lane & 15, g4 = lane >> 4;
  const int r0 = blockIdx.x * 16, nr = min(16, c.R - r0), E = c.r.experts;
  const size_t row = (size_t)(r0 + min(c16, nr - 1)) * c.ld + 8 * g4;
  const float* x = H16 ? nullptr : c.x + row;
  const T* xh = (const T*)c.h + row;
  f32x4 acc[NE];
#pragma unroll
  for (int t = 0; t < NE; ++t) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  constexpr int KU = NE <= 2 ? 4 : (NE <= 4 ? 2 : 1);               // k steps whose loads are in flight together
  for (int k0 = wave * 32; k0 < c.ld; k0 += KU * RTW * 32) {
    float v[H16 ? 1 : KU][8];
    u32x4 vh[H16 ? KU : 1], b[KU][NE];
#pragma unroll
    for (int u = 0; u < KU; ++u) {
      const int k = min(k0 + u * RTW * 32, c.ld - 32);               // (steps beyond the row: loaded, not used)
      if constexpr (H16) vh[u] = *(const u32x4*)(xh + k);
      else load8f<float>(x + k, v[u]);
#pragma unroll
      for (int t = 0; t < NE; ++t) b[u][t] = *(const u32x4*)((const T*)c.router + (size_t)min(t * 16 + c16, E - 1) * c.ld + k + 8 * g4);
    }
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int u = 0; u < KU; ++u)
      if (k0 + u * RTW * 32 < c.ld) {
        if constexpr (H16) {
#pragma unroll
          for (int t = 0; t < NE; ++t) acc[t] = mfma16<T>(vh[u], b[u][t], acc[t]);
        } else {
          T hi[8], lo[8];
#pragma unroll
          for (int i = 0; i < 8; ++i) { hi[i] = (T)v[u][i]; lo[i] = (T)(v[u][i] - (float)hi[i]); }
          const u32x4 ah = __builtin_bit_cast(u32x4, hi), al = __builtin_bit_cast(u32x4, lo);
#pragma unroll
          for (int t = 0; t < NE; ++t) {
            acc[t] = mfma16<T>(ah, b[u][t], acc[t]);
            acc[t] = mfma16<T>(al, b[u][t], acc[t]);
          }
        }
      }
  }
#pragma unroll
  for (int t = 0; t < NE; ++t) *(f32x4*)(sm + ((wave * NE + t) * 64 + lane) * 4) = acc[t];
  __syncthreads();
  // logits: lane (e & 15, m >> 2) of tile e >> 4 holds row m = 4 g4 + r
  constexpr int EP = 16 * NE, PER = (16 * EP + RTW * 64 - 1) / (RTW * 64);
  float z[PER];
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int idx = i * RTW * 64 + tid, m = min(idx / EP, 15), e = idx % EP;
    float s = 0.f;
#pragma unroll
    for (int w = 0; w < RTW; ++w) s += sm[((w * NE + (e >> 4)) * 64 + (m >> 2) * 16 + (e & 15)) * 4 + (m & 3)];
    z[i] = c.r.bias != nullptr ? s + c.r.bias[min(e, E - 1)] : s;
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < PER; ++i) { const int idx = i * RTW * 64 + tid; if (idx < 16 * EP) sm[idx] = z[i]; }
  __syncthreads();
  const int top = c.r.top;
  float* sw = sm + 16 * EP + wave * route_lds_floats(c.r);
  int* sel = (int*)(sm + 16 * EP + RTW * route_lds_floats(c.r));       // [16][top]
  int* cnt = sel + 16 * top;                                          // [E] of this workgroup, then the places in front of them
  for (int e = tid; e < E; e += RTW * 64) cnt[e] = 0;
  for (int m = wave; m < nr; m += RTW) route_wave(sm + m * EP, c.r, sel + m * top, sw, c.ids + (size_t)(r0 + m) * top, c.wts + (size_t)(r0 + m) * top);
  __syncthreads();
  // places among the expert's slots (their order does not matter): one global addition per expert and workgroup
  constexpr int NI = (16 * MOE_MAX_TOP + RTW * 64 - 1) / (RTW * 64);
  int at[NI];
#pragma unroll
  for (int i = 0; i < NI; ++i) { const int idx = i * RTW * 64 + tid; at[i] = idx < nr * top ? atomicAdd(&cnt[sel[idx]], 1) : 0; }
  __syncthreads();
  for (int e = tid; e < E; e += RTW * 64) cnt[e] = cnt[e] > 0 ? atomicAdd(&c.counts[e], cnt[e]) : 0;
  __syncthreads();
#pragma unroll
  for (int i = 0; i < NI; ++i) { const int idx = i * RTW * 64 + tid; if (idx < nr * top) c.counts[E + (size_t)r0 * top + idx] = cnt[sel[idx]] + at[i]; }
}

template <typename T, bool H16>
int route_rows(const MoeCall& c, hipStream_t st) {
  const int ne = (c.r.experts + 15) / 16;
  auto go = [&](auto k, int NE, int RTW) -> int {
    const size_t part = (size_t)RTW * NE * 1024,
                 pick = ((size_t)16 * 16 * NE + RTW * route_lds_floats(c.r) + 16 * c.r.top + c.r.experts) * sizeof(float);
    const size_t lds = std::max(part, pick);
    if (lds > 65536) MI_HIP(hipFuncSetAttribute((const void*)k, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    hipLaunchKernelGGL(k, dim3((c.R + 15) / 16), dim3(RTW * 64), lds, st, c);
    MI_HIP(hipGetLastError());
    return MI_OK;
  };
  if (ne <= 1) return go(route_kernel<T, 1, 16, H16>, 1, 16);
  if (ne <= 2) return go(route_kernel<T, 2, 16, H16>, 2, 16);
  if (ne <= 4) return go(route_kernel<T, 4, 16, H16>, 4, 16);
  if (ne <= 8) return go(route_kernel<T, 8, 16, H16>, 8, 16);
  return go(route_kernel<T, 16, 8, H16>, 16, 8);             // (route_fused: at most ROUTE_MFMA_EXPERTS)
}
template <typename T>
int route_at(const MoeCall& c, hipStream_t st) { return c.x != nullptr ? route_rows<T, false>(c, st) : route_rows<T, true>(c, st); }
constexpr int ROUTE_MFMA_EXPERTS = 256;

// ---- plan: the slots sorted by expert, and the tile table ------------------------------------------------------------------
// words: [0] tiles, [8 ..) tiles of four words (expert, first place, places, 0), then slot and token of every place
inline int plan_tiles(int R, int experts, int top, int shared, int tile) {
  return R * top / tile + experts + (shared ? (R + tile - 1) / tile : 0);
}
// places per tile: the large tile where an expert fills at least most of one on average
constexpr int MOE_LARGE = 160;
inline int tile_of(const MoeCall& c) {
  const bool deep = c.ld >= 128 && c.ffp >= 128 && (c.sffp == 0 || c.sffp >= 128);
  return deep && (size_t)c.R * c.r.top >= (size_t)MOE_LARGE * c.r.experts ? 256 : 128;
}
// counts of a router that does not count (launch_post_norm's): one workgroup
__global__ __launch_bounds__(1024) void moe_count_kernel(MoeCall c) {
  __shared__ int cnt[MOE_MAX_EXPERTS];
  const int tid = threadIdx.x, E = c.r.experts, n = c.R * c.r.top;
  for (int e = tid; e < E; e += 1024) cnt[e] = 0;
  __syncthreads();
  for (int i = tid; i < n; i += 1024) c.counts[E + i] = atomicAdd(&cnt[min(max(c.ids[i], 0), E - 1)], 1);
  __syncthreads();
  for (int e = tid; e < E; e += 1024) c.counts[e] = cnt[e];
}

// grid: PLAN_SLOTS slots per workgroup (every one makes the running sums for itself); the first also writes the table
constexpr int PLAN_SLOTS = 4096;
__global__ __launch_bounds__(1024) void moe_plan_kernel(MoeCall c, int max_tiles, int tile) {
  __shared__ int cnt[MOE_MAX_EXPERTS], start[MOE_MAX_EXPERTS], tile0[MOE_MAX_EXPERTS + 1];
  const int tid = threadIdx.x, E = c.r.experts, n = c.R * c.r.top, shared = c.sffp > 0, ns = shared ? (c.R + tile - 1) / tile : 0;
  int32_t* tiles = c.plan + 8;
  int32_t* slot = tiles + 4 * max_tiles;
  int32_t* token = slot + n + (shared ? c.R : 0);
  for (int e = tid; e < E; e += 1024) cnt[e] = c.counts[e];
  __syncthreads();
  if (tid < 64) {                                      // running sums of places and tiles, 64 experts at a time
    int p0 = 0, t0 = ns;                               // (the shared expert's tiles first: it is usually the widest)
    for (int b = 0; b < E; b += 64) {
      const int e = b + tid, k = e < E ? cnt[e] : 0, t = (k + tile - 1) / tile;
      int p = k, q = t;
      for (int o = 1; o < 64; o *= 2) {
        const int pu = __shfl_up(p, o, 64), qu = __shfl_up(q, o, 64);
        if (tid >= o) { p += pu; q += qu; }
      }
      if (e < E) { start[e] = p0 + p - k; tile0[e] = t0 + q - t; }
      p0 += __shfl(p, 63, 64);
      t0 += __shfl(q, 63, 64);
    }
    if (tid == 0) tile0[E] = t0;
  }
  __syncthreads();
  if (blockIdx.x == 0) {
    for (int e = tid; e < E; e += 1024)
      for (int i = 0, k = 0; k < cnt[e]; ++i, k += tile) {
        int32_t* t = tiles + 4 * (tile0[e] + i);
        t[0] = e; t[1] = start[e] + k; t[2] = min(tile, cnt[e] - k); t[3] = 0;
      }
    for (int i = tid; i < ns; i += 1024) {
      int32_t* t = tiles + 4 * i;
      t[0] = E; t[1] = n + i * tile; t[2] = min(tile, c.R - i * tile); t[3] = 0;
    }
    if (tid == 0) c.plan[0] = tile0[E];
  }
  const int end = min(n + (shared ? c.R : 0), (int)(blockIdx.x + 1) * PLAN_SLOTS);
  for (int i = blockIdx.x * PLAN_SLOTS + tid; i < end; i += 1024) {
    const int p = i < n ? start[min(max(c.ids[i], 0), E - 1)] + c.counts[E + i] : i;
    slot[p] = i;
    token[p] = i < n ? i / c.r.top : i - n;
  }
}

// ---- streaming form -------------------------------------------------------------------------------------------------------
// the slots of expert e into list[], their number returned to every thread; their order does not matter
__device__ __forceinline__ int collect(const MoeCall& c, int e, int* list, int* n_sh) {
  const int tid = threadIdx.x, n = c.R * c.r.top;
  if (e == c.r.experts) {
    for (int i = tid; i < c.R; i += 256) list[i] = n + i;
    __syncthreads();
    return c.R;
  }
  if (tid == 0) *n_sh = 0;
  __syncthreads();
  for (int i = tid; i < n; i += 256)
    if (c.ids[i] == e) { const int p = atomicAdd(n_sh, 1); if (p < MOE_STREAM_ROWS) list[p] = i; }     // (at most one slot per token)
  __syncthreads();
  return min(*n_sh, MOE_STREAM_ROWS);
}

constexpr int MOE_KU = 8;      // k steps of 32 whose loads are in flight together

// one strip (NTW tiles of 16 weight rows, wt[]: their tile numbers) times up to 16 MT rows of x; K split over the four waves,
// whose partial tiles end up in `red` [4][NTW][MT][64][4]
template <typename T, int NTW, int MT>
__device__ __forceinline__ void strip_product(const char* w, const int (&wt)[NTW], int ksteps, const T* const (&xrow)[MT], float* red) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, g4 = lane >> 4;
  f32x4 acc[NTW][MT];
#pragma unroll
  for (int t = 0; t < NTW; ++t)
#pragma unroll
    for (int m = 0; m < MT; ++m) acc[t][m] = f32x4{0.f, 0.f, 0.f, 0.f};
  const char* wp[NTW];
#pragma unroll
  for (int t = 0; t < NTW; ++t) wp[t] = w + (size_t)wt[t] * ksteps * 1024 + lane * 16;
  for (int s0 = wave; s0 < ksteps; s0 += 4 * MOE_KU) {
    u32x4 wf[MOE_KU][NTW], xf[MOE_KU][MT];
#pragma unroll
    for (int u = 0; u < MOE_KU; ++u) {
      const int s = min(s0 + 4 * u, ksteps - 1);
#pragma unroll
      for (int t = 0; t < NTW; ++t) wf[u][t] = *(const u32x4*)(wp[t] + (size_t)s * 1024);
#pragma unroll
      for (int m = 0; m < MT; ++m) xf[u][m] = *(const u32x4*)(xrow[m] + 32 * s + 8 * g4);
    }
#pragma unroll
    for (int u = 0; u < MOE_KU; ++u)
      if (s0 + 4 * u < ksteps) {
#pragma unroll
        for (int t = 0; t < NTW; ++t)
#pragma unroll
          for (int m = 0; m < MT; ++m) acc[t][m] = mfma16<T>(wf[u][t], xf[u][m], acc[t][m]);
      }
  }
#pragma unroll
  for (int t = 0; t < NTW; ++t)
#pragma unroll
    for (int m = 0; m < MT; ++m) *(f32x4*)(red + (((wave * NTW + t) * MT + m) * 64 + lane) * 4) = acc[t][m];
  __syncthreads();
}

// sum over the waves of tile (t, m), this lane's four values: weight rows 4 g4 + r, slot column c16
template <int NTW, int MT>
__device__ __forceinline__ f32x4 strip_sum(const float* red, int t, int m) {
  const int lane = threadIdx.x & 63;
  f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int w = 0; w < 4; ++w) s += *(const f32x4*)(red + (((w * NTW + t) * MT + m) * 64 + lane) * 4);
  return s;
}

// grid (strips, experts + shared): mid[slot] = glu(W_gate h, W_up h).  A strip: one gate tile and its up tile
template <typename T, int MT>
__global__ __launch_bounds__(256) void moe_stream_up_kernel(MoeCall c) {
  __shared__ int list[MOE_STREAM_ROWS];
  __shared__ int n_sh;
  __shared__ __attribute__((aligned(16))) float red[4 * 2 * MT * 256];
  const int e = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c16 = lane & 15, g4 = lane >> 4;
  const bool sh = e == c.r.experts;
  const int ffp = sh ? c.sffp : c.ffp, strip = blockIdx.x;
  if (strip * 16 >= ffp) return;
  const int n = collect(c, e, list, &n_sh), ntok = c.R * c.r.top;
  const char* W = (const char*)(sh ? c.sgu.w : c.gu.w);
  const int base = sh ? 0 : e * 2 * (ffp / 16);
  const int wt[2] = {base + strip, base + ffp / 16 + strip};
  for (int m0 = 0; m0 < n; m0 += 16 * MT) {
    const T* xrow[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      const int s = list[min(m0 + 16 * m + c16, n - 1)];
      xrow[m] = (const T*)c.h + (size_t)(s < ntok ? s / c.r.top : s - ntok) * c.ld;
    }
    strip_product<T, 2, MT>(W, wt, c.ld / 32, xrow, red);
    for (int m = wave; m < MT; m += 4) {
      const f32x4 g = strip_sum<2, MT>(red, 0, m), u = strip_sum<2, MT>(red, 1, m);
      const int i = m0 + 16 * m + c16;
      if (i < n) {
        T o[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) o[r] = from_f32<T>(glu_f(c.glu, g[r], u[r]));
        *(uint2*)((T*)c.mid + (size_t)list[i] * c.lda + strip * 16 + 4 * g4) = __builtin_bit_cast(uint2, o);
      }
    }
    __syncthreads();
  }
}

// grid (strips, experts + shared): out[slot] = W_down mid[slot].  A strip: two tiles
template <typename T, int MT>
__global__ __launch_bounds__(256) void moe_stream_down_kernel(MoeCall c) {
  __shared__ int list[MOE_STREAM_ROWS];
  __shared__ int n_sh;
  __shared__ __attribute__((aligned(16))) float red[4 * 2 * MT * 256];
  const int e = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c16 = lane & 15, g4 = lane >> 4;
  const bool sh = e == c.r.experts;
  const int ffp = sh ? c.sffp : c.ffp, strip = blockIdx.x;
  const int n = collect(c, e, list, &n_sh);
  const char* W = (const char*)(sh ? c.sdn.w : c.dn.w);
  const int base = (sh ? 0 : e * (c.ld / 16)) + 2 * strip;
  const int wt[2] = {base, base + 1};                  // (ld is a multiple of 64)
  for (int m0 = 0; m0 < n; m0 += 16 * MT) {
    const T* xrow[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) xrow[m] = (const T*)c.mid + (size_t)list[min(m0 + 16 * m + c16, n - 1)] * c.lda;
    strip_product<T, 2, MT>(W, wt, ffp / 32, xrow, red);
    for (int tm = wave; tm < 2 * MT; tm += 4) {
      const int t = tm & 1, m = tm >> 1, i = m0 + 16 * m + c16;
      const f32x4 v = strip_sum<2, MT>(red, t, m);
      if (i < n) {
        T o[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) o[r] = from_f32<T>(v[r]);
        *(uint2*)((T*)c.out + (size_t)list[i] * c.ld + strip * 32 + t * 16 + 4 * g4) = __builtin_bit_cast(uint2, o);
      }
    }
    __syncthreads();
  }
}

template <typename T, bool UP>
int stream_at(const MoeCall& c, hipStream_t st) {
  const int ny = c.r.experts + (c.sffp > 0 ? 1 : 0);
  const dim3 grid(UP ? std::max(c.ffp, c.sffp) / 16 : c.ld / 32, ny);
  if constexpr (UP) {
    if (c.R <= 16) hipLaunchKernelGGL((moe_stream_up_kernel<T, 1>), grid, dim3(256), 0, st, c);
    else hipLaunchKernelGGL((moe_stream_up_kernel<T, 2>), grid, dim3(256), 0, st, c);
  } else {
    if (c.R <= 16) hipLaunchKernelGGL((moe_stream_down_kernel<T, 1>), grid, dim3(256), 0, st, c);
    else hipLaunchKernelGGL((moe_stream_down_kernel<T, 2>), grid, dim3(256), 0, st, c);
  }
  MI_HIP(hipGetLastError());
  return MI_OK;
}

// ---- generic form: grid (slots, strips of 64 rows), 4 waves of 16 rows each; row-major weights -----------------------------
template <typename T, bool UP>
__global__ __launch_bounds__(256) void moe_generic_kernel(MoeCall c) {
  extern __shared__ __attribute__((aligned(16))) float xs[];      // the slot's input row
  const int slot = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, n = c.R * c.r.top;
  const bool sh = slot >= n;
  const int e = sh ? 0 : min(max(c.ids[slot], 0), c.r.experts - 1), ffp = sh ? c.sffp : c.ffp;
  const int rows = UP ? ffp : c.ld, K = UP ? c.ld : ffp, r0 = blockIdx.y * 64;
  if (r0 >= rows) return;
  const T* src = UP ? (const T*)c.h + (size_t)(sh ? slot - n : slot / c.r.top) * c.ld : (const T*)c.mid + (size_t)slot * c.lda;
  for (int k = threadIdx.x; k < K; k += 256) xs[k] = to_f32(src[k]);
  __syncthreads();
  const T* w = (const T*)(UP ? (sh ? c.sgu.w : c.gu.w) : (sh ? c.sdn.w : c.dn.w)) + (size_t)e * (UP ? 2 * ffp : c.ld) * K;
  auto dot = [&](int row) {
    const T* p = w + (size_t)row * K;
    float a = 0.f;
    for (int k = lane; k < K; k += 64) a = fmaf(to_f32(p[k]), xs[k], a);
    return wave_sum(a);
  };
  for (int i = wave; i < 64 && r0 + i < rows; i += 4) {
    const int row = r0 + i;
    float v = dot(row);
    if constexpr (UP) v = glu_f(c.glu, v, dot(ffp + row));
    if (lane == 0) {
      if constexpr (UP) ((T*)c.mid)[(size_t)slot * c.lda + row] = from_f32<T>(v);
      else ((T*)c.out)[(size_t)slot * c.ld + row] = from_f32<T>(v);
    }
  }
}

template <typename T, bool UP>
int generic_at(const MoeCall& c, hipStream_t st) {
  const int slots = c.R * c.r.top + (c.sffp > 0 ? c.R : 0);
  const size_t lds = (size_t)(UP ? c.ld : c.lda) * sizeof(float);
  if (lds > 160 * 1024 - 1024) return fail(MI_ERR_UNSUPPORTED, "moe: row too wide for the LDS");
  auto k = moe_generic_kernel<T, UP>;
  if (lds > 65536) MI_HIP(hipFuncSetAttribute((const void*)k, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
  hipLaunchKernelGGL(k, dim3(slots, ((UP ? std::max(c.ffp, c.sffp) : c.ld) + 63) / 64), dim3(256), lds, st, c);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

}  // namespace

size_t moe_plan_ints(int R, const RouteArgs& r, int shared) {
  return 8 + 4 * (size_t)plan_tiles(R, r.experts, r.top, shared, 128) + 2 * ((size_t)R * r.top + (shared ? R : 0));
}

// the matrix-core forms read tile-major 16-bit weights
bool moe_mfma_supported(const MoeCall& c) {
  return (c.act == MI_BF16 || c.act == MI_F16) && c.gu.layout == 1 && c.dn.layout == 1 && c.ffp % 64 == 0 && c.sffp % 64 == 0 &&
         (c.sffp == 0 || (c.sgu.layout == 1 && c.sdn.layout == 1));
}

bool route_fused(int act, int rows, int experts) { return act == MI_F32 || rows < MOE_STREAM_ROWS || experts > ROUTE_MFMA_EXPERTS; }

int launch_route(const MoeCall& c, hipStream_t st) {
  if (c.r.experts > ROUTE_MFMA_EXPERTS) return fail(MI_ERR_UNSUPPORTED, "route: too many experts");
  if (c.act == MI_BF16) return route_at<bf16>(c, st);
  if (c.act == MI_F16) return route_at<f16>(c, st);
  return fail(MI_ERR_UNSUPPORTED, "route: 16-bit models only");
}

namespace {

enum : int { FORM_GENERIC, FORM_STREAM, FORM_TILES };
int form_of(const MoeCall& c, int& form) {
  if (c.r.experts < 1 || c.r.experts > MOE_MAX_EXPERTS || c.r.top < 1 || c.r.top > MOE_MAX_TOP || c.ld % 64 != 0)
    return fail(MI_ERR_INVALID, "moe: sizes out of range");
  if (c.act != MI_F32 && c.act != MI_BF16 && c.act != MI_F16) return fail(MI_ERR_INVALID, "moe: bad dtype");
  form = FORM_GENERIC;
  if (moe_mfma_supported(c)) form = c.R <= MOE_STREAM_ROWS ? FORM_STREAM : FORM_TILES;
  else if (c.gu.layout != 0 || c.dn.layout != 0 || (c.sffp > 0 && (c.sgu.layout != 0 || c.sdn.layout != 0)))
    return fail(MI_ERR_INVALID, "moe: mixed weight layouts");
  return MI_OK;
}

template <bool UP>
int experts_at(const MoeCall& c, hipStream_t st) {
  int form = FORM_GENERIC;
  MI_TRY(form_of(c, form));
  if (form == FORM_GENERIC) return c.act == MI_F32 ? generic_at<float, UP>(c, st) : (c.act == MI_BF16 ? generic_at<bf16, UP>(c, st) : generic_at<f16, UP>(c, st));
  if (form == FORM_STREAM) return c.act == MI_BF16 ? stream_at<bf16, UP>(c, st) : stream_at<f16, UP>(c, st);
  const int shared = c.sffp > 0 ? 1 : 0, n = c.R * c.r.top, tile = tile_of(c), max_tiles = plan_tiles(c.R, c.r.experts, c.r.top, shared, tile);
  const int32_t* slot = c.plan + 8 + 4 * max_tiles;
  const int32_t* token = slot + n + (shared ? c.R : 0);
  GroupedGemm g{};
  g.tiles = c.plan; g.max_tiles = max_tiles; g.tile = tile; g.groups = c.r.experts; g.act = c.act; g.swiglu = UP; g.glu = c.glu;
  if (UP) {
    g.x = c.h; g.ldx = c.ld; g.x_rows = token; g.out = c.mid; g.ldo = c.lda;
    g.W = c.gu; g.rows = 2 * c.ffp; g.last = shared ? c.sgu : LinearW{};
  } else {
    g.x = c.mid; g.ldx = c.lda; g.out = c.out; g.ldo = c.ld; g.out_rows = slot;
    g.W = c.dn; g.rows = c.ld; g.last = shared ? c.sdn : LinearW{};
  }
  return launch_gemm_grouped(g, st);
}

}  // namespace

int launch_moe_plan(const MoeCall& c, hipStream_t st) {
  int form = FORM_GENERIC;
  MI_TRY(form_of(c, form));
  if (form != FORM_TILES) return MI_OK;
  if (route_fused(c.act, c.R, c.r.experts)) {
    hipLaunchKernelGGL(moe_count_kernel, dim3(1), dim3(1024), 0, st, c);
    MI_HIP(hipGetLastError());
  }
  const int shared = c.sffp > 0 ? 1 : 0, slots = c.R * (c.r.top + shared);
  hipLaunchKernelGGL(moe_plan_kernel, dim3((slots + PLAN_SLOTS - 1) / PLAN_SLOTS), dim3(1024), 0, st, c,
                     plan_tiles(c.R, c.r.experts, c.r.top, shared, tile_of(c)), tile_of(c));
  MI_HIP(hipGetLastError());
  return MI_OK;
}
int launch_moe_up(const MoeCall& c, hipStream_t st) { return experts_at<true>(c, st); }
int launch_moe_down(const MoeCall& c, hipStream_t st) { return experts_at<false>(c, st); }

}  // namespace mi
