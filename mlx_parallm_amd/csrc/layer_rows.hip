// layer_rows.hip -- row-wise steps of layer-list models: embedding + positions + first norm, per-layer token input + the norm
// in front of the next layer, residual update of post- and pre-norm blocks (the latter with several streams).  The residual stream
// is float32; the normed rows that feed the matrix products are in the activation dtype.
#include <algorithm>
#include <cmath>
#include <type_traits>

#include "layer_rows.h"

namespace mi {

namespace {

using namespace rows;

template <typename T, int NT>
__global__ __launch_bounds__(NT) void embed_pos_kernel(EmbedPosCall c) {
  __shared__ float red[NT / 64];
  const int r = blockIdx.x, streams = max(c.streams, 1);
  const int tok = min(max(c.tokens[r], 0), c.vocab - 1);
  const TokenAt at = token_at(c.t, r);
  const int pos = at.pos;
  const T* src = (const T*)c.table + (size_t)tok * c.width;
  const T* pair = nullptr;
  if (c.pair.table != nullptr) {
    int row = c.pair.buckets;
    if (pos > 0) {
      const int before = min(max(at.t > 0 ? c.tokens[r - 1] : c.pair.prev[at.row], 0), c.vocab - 1);
      row = (int)(((uint64_t)before * (uint64_t)c.pair.mul_prev + (uint64_t)tok * (uint64_t)c.pair.mul_cur) % (uint64_t)c.pair.buckets);
    }
    pair = (const T*)c.pair.table + (size_t)row * c.width;
  }
  float fin = (float)streams;                        // what is read of the streams is fin x
  if (c.in != nullptr) {
    fin = 0.f;
    for (int s = 0; s < streams; ++s) fin += c.in[s];
  }
  float* x = c.x + (size_t)r * streams * c.ld;
  float ss[1] = {0.f};
  for (int k = 2 * threadIdx.x; k < c.ld; k += 2 * NT) {        // (ld is even)
    float2 v = {0.f, 0.f};
    if (k < c.width) {
      v.x = to_f32(src[k]) * c.scale;
      if (k + 1 < c.width) v.y = to_f32(src[k + 1]) * c.scale;
      if (c.freq != nullptr) {
        // the angle is reduced in double precision, the functions taken in single
        const double a = (double)pos * c.freq[k >> 1];
        const float f = (float)(a - 6.283185307179586 * rint(a * 0.15915494309189535));
        v.x += sinf(f);
        if (k + 1 < c.width) v.y += cosf(f);
      }
      if (pair != nullptr) {
        v.x += to_f32(pair[k]);
        if (k + 1 < c.width) v.y += to_f32(pair[k + 1]);
      }
      ss[0] += v.x * v.x + v.y * v.y;
    }
    for (int s = 0; s < streams; ++s) *(float2*)(x + (size_t)s * c.ld + k) = v;
  }
  T* h = (T*)c.h + (size_t)r * c.ld;
  if (c.norm.w == nullptr) {
    for (int k = 2 * threadIdx.x; k < c.ld; k += 2 * NT)
#pragma unroll
      for (int j = k; j < k + 2; ++j) h[j] = from_f32<T>(x[j]);
    return;
  }
  block_sum<NT, 1>(ss, red);
  const float rs = fin / sqrtf(ss[0] * fin * fin / (float)c.width + c.norm.eps);
  for (int k = 2 * threadIdx.x; k < c.ld; k += 2 * NT)          // (each thread reads what it wrote)
#pragma unroll
    for (int j = k; j < k + 2; ++j)
      h[j] = j < c.width ? from_f32<T>(x[j] * rs * c.norm.w[j * c.norm.stride]) : from_f32<T>(0.f);
}

// RB rows per workgroup: the gate and projection weights are read once for all of them.
template <typename T, int NT, int RB>
__global__ __launch_bounds__(NT) void side_norm_kernel(SideNormCall c) {
  extern __shared__ float smem[];
  float* xs = smem;                          // [RB][ld]
  float* ys = xs + (size_t)RB * c.ld;        // [RB][ld]
  float* gs = ys + (size_t)RB * c.ld;        // [RB][dim]
  __shared__ float red[(NT / 64) * RB];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  constexpr int NW = NT / 64;
  const int r0 = blockIdx.x * RB, nr = min(RB, c.rows - r0);
  const int n4 = c.ld / 4;
#pragma unroll
  for (int b = 0; b < RB; ++b) {
    const float4* src = (const float4*)(c.x + (size_t)(r0 + min(b, nr - 1)) * c.ld);
    for (int i = tid; i < n4; i += NT) ((float4*)(xs + (size_t)b * c.ld))[i] = src[i];
  }
  __syncthreads();
  float ss[RB];
  if (c.dim > 0) {
    // gate: a wave takes JB outputs at a time, its lanes split the row
    constexpr int JB = 4;
    for (int j0 = wave * JB; j0 < c.dim; j0 += NW * JB) {
      float acc[JB][RB];
#pragma unroll
      for (int j = 0; j < JB; ++j)
#pragma unroll
        for (int b = 0; b < RB; ++b) acc[j][b] = 0.f;
      for (int k = lane * 8; k < c.ld; k += 512) {
        float w[JB][8];
#pragma unroll
        for (int j = 0; j < JB; ++j) load8f<T>((const T*)c.gate + (size_t)min(j0 + j, c.dim - 1) * c.ld + k, w[j]);
#pragma unroll
        for (int b = 0; b < RB; ++b) {
          float xv[8];
          load8f<float>(xs + (size_t)b * c.ld + k, xv);
#pragma unroll
          for (int j = 0; j < JB; ++j)
#pragma unroll
            for (int i = 0; i < 8; ++i) acc[j][b] = fmaf(w[j][i], xv[i], acc[j][b]);
        }
      }
#pragma unroll
      for (int j = 0; j < JB; ++j)
#pragma unroll
        for (int b = 0; b < RB; ++b) {
          const float z = wave_sum(acc[j][b]);
          if (lane == 0 && j0 + j < c.dim) {
            const int tok = min(max(c.tokens[r0 + min(b, nr - 1)], 0), c.vocab - 1);
            gs[b * c.dim + j0 + j] = gelu_tanh_f(z) * to_f32(((const T*)c.table)[(size_t)tok * c.table_ld + c.slice + j0 + j]);
          }
        }
    }
    __syncthreads();
#pragma unroll
    for (int b = 0; b < RB; ++b) ss[b] = 0.f;
    for (int i = tid; i < n4; i += NT) {
      float4 y[RB];
#pragma unroll
      for (int b = 0; b < RB; ++b) y[b] = float4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
      for (int j = 0; j < c.dim; ++j) {
        const float4 w = load4f<T>((const T*)c.proj_t + (size_t)j * c.ld + 4 * i);
#pragma unroll
        for (int b = 0; b < RB; ++b) {
          const float g = gs[b * c.dim + j];
          y[b].x = fmaf(w.x, g, y[b].x); y[b].y = fmaf(w.y, g, y[b].y);
          y[b].z = fmaf(w.z, g, y[b].z); y[b].w = fmaf(w.w, g, y[b].w);
        }
      }
#pragma unroll
      for (int b = 0; b < RB; ++b) {
        ((float4*)(ys + (size_t)b * c.ld))[i] = y[b];
        ss[b] += y[b].x * y[b].x + y[b].y * y[b].y + y[b].z * y[b].z + y[b].w * y[b].w;
      }
    }
    block_sum<NT, RB>(ss, red);
    float rs[RB];
#pragma unroll
    for (int b = 0; b < RB; ++b) rs[b] = 1.0f / sqrtf(ss[b] / (float)c.width + c.side_eps);
#pragma unroll
    for (int b = 0; b < RB; ++b) {
      for (int k = tid; k < c.width; k += NT) {
        const float v = xs[(size_t)b * c.ld + k] + ys[(size_t)b * c.ld + k] * rs[b] * c.side_w[k];
        xs[(size_t)b * c.ld + k] = v;
        if (b < nr) c.x[(size_t)(r0 + b) * c.ld + k] = v;
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int b = 0; b < RB; ++b) {
    ss[b] = 0.f;
    for (int k = tid; k < c.width; k += NT) { const float v = xs[(size_t)b * c.ld + k]; ss[b] += v * v; }
  }
  block_sum<NT, RB>(ss, red);
#pragma unroll
  for (int b = 0; b < RB; ++b) {
    if (b >= nr) break;
    const float rn = 1.0f / sqrtf(ss[b] / (float)c.width + c.norm.eps);
    T* h = (T*)c.h + (size_t)(r0 + b) * c.ld;
    for (int k = tid; k < c.ld; k += NT)
      h[k] = k < c.width ? from_f32<T>(xs[(size_t)b * c.ld + k] * rn * c.norm.w[k * c.norm.stride]) : from_f32<T>(0.f);
  }
}

// ---- the same on the matrix cores: 16 rows per workgroup, 8 waves (16-bit weights; calls of many rows) ------------------
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

constexpr int SNW = 8;
// NTW: 16-column tiles of the row per wave (ld <= 128 NTW), 0: any number.  The residual itself stays float32: only the gate's operand is 16-bit.
template <typename T, int NTW>
__global__ __launch_bounds__(SNW * 64) void side_norm_mfma_kernel(SideNormCall c) {
  extern __shared__ __attribute__((aligned(16))) unsigned char sm[];
  const int dp = (c.dim + 31) & ~31, ldx = c.ld + 8, ldg = dp + 8, ndt = dp / 16;
  T* xs = (T*)sm;                                    // [16][ldx], then the waves' partial gate tiles [SNW][ndt][64][4] floats
  float* pt = (float*)sm;
  __shared__ __attribute__((aligned(16))) T gs[16 * (128 + 8)];
  __shared__ float red[2][SNW][16];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c16 = lane & 15, g4 = lane >> 4;
  const int r0 = blockIdx.x * 16, nr = min(16, c.rows - r0), ntiles = c.ld / 16;
  for (int i = tid; i < 16 * (c.ld / 4); i += SNW * 64) {
    const int m = i / (c.ld / 4), k = i % (c.ld / 4) * 4;
    const float4 v = *(const float4*)(c.x + (size_t)(r0 + min(m, nr - 1)) * c.ld + k);
    T o[4] = {(T)v.x, (T)v.y, (T)v.z, (T)v.w};
    *(uint2*)(xs + m * ldx + k) = __builtin_bit_cast(uint2, o);
  }
  __syncthreads();
  // gate: every wave takes every eighth k step of all tiles
  f32x4 acc[8];
#pragma unroll
  for (int t = 0; t < 8; ++t) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k = wave * 32; k < c.ld; k += SNW * 32) {
    const u32x4 a = *(const u32x4*)(xs + c16 * ldx + k + 8 * g4);
#pragma unroll
    for (int t = 0; t < 8; ++t)
      if (t < ndt) acc[t] = mfma16<T>(a, *(const u32x4*)((const T*)c.gate + (size_t)min(t * 16 + c16, c.dim - 1) * c.ld + k + 8 * g4), acc[t]);
  }
  __syncthreads();
#pragma unroll
  for (int t = 0; t < 8; ++t)
    if (t < ndt) *(f32x4*)(pt + ((wave * ndt + t) * 64 + lane) * 4) = acc[t];
  __syncthreads();
  for (int i = tid; i < 16 * dp; i += SNW * 64) {
    const int m = i / dp, j = i % dp, el = (m >> 2) * 16 + (j & 15);
    float z = 0.f;
#pragma unroll
    for (int w = 0; w < SNW; ++w) z += pt[((w * ndt + (j >> 4)) * 64 + el) * 4 + (m & 3)];
    float g = 0.f;
    if (j < c.dim) {
      const int tok = min(max(c.tokens[r0 + min(m, nr - 1)], 0), c.vocab - 1);
      g = gelu_tanh_f(z) * to_f32(((const T*)c.table)[(size_t)tok * c.table_ld + c.slice + j]);
    }
    gs[m * ldg + j] = (T)g;
  }
  __syncthreads();
  // one 16-column tile of y = proj g
  auto y_tile = [&](int i) {
    const int nt = min(wave + SNW * i, ntiles - 1);
    const T* w = (const T*)c.proj_p + (size_t)(nt * 16 + c16) * dp + 8 * g4;
    f32x4 v = {0.f, 0.f, 0.f, 0.f};
    for (int k = 0; k < dp; k += 32) v = mfma16<T>(*(const u32x4*)(gs + c16 * ldg + k + 8 * g4), *(const u32x4*)(w + k), v);
    return v;
  };
  float ss[4] = {0.f, 0.f, 0.f, 0.f}, rs[4];
  auto row_sums = [&](int which) {                   // ss[r] of row 4 g4 + r over the row's columns: 16 lanes, then the waves
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float v = row16_sum(ss[r]);
      if (c16 == 0) red[which][wave][4 * g4 + r] = v;
    }
    __syncthreads();
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      ss[r] = 0.f;
#pragma unroll
      for (int w = 0; w < SNW; ++w) ss[r] += red[which][w][4 * g4 + r];
    }
  };
  // the residual at one place, with the token input added
  auto add_x = [&](f32x4 v, int col) {
    const float w = col < c.width ? c.side_w[col] : 0.f;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float x = col < c.ld ? c.x[(size_t)(r0 + min(4 * g4 + r, nr - 1)) * c.ld + col] : 0.f;
      v[r] = fmaf(v[r] * rs[r], w, x);
      ss[r] += v[r] * v[r];
    }
    return v;
  };
  auto inv_rms = [&](float eps) {
#pragma unroll
    for (int r = 0; r < 4; ++r) { rs[r] = 1.0f / sqrtf(ss[r] / (float)c.width + eps); ss[r] = 0.f; }
  };
  if constexpr (NTW > 0) {                           // the row stays in registers
    f32x4 y[NTW];
#pragma unroll
    for (int i = 0; i < NTW; ++i) {
      y[i] = y_tile(i);
      if (wave + SNW * i < ntiles) {
#pragma unroll
        for (int r = 0; r < 4; ++r) ss[r] += y[i][r] * y[i][r];
      }
    }
    row_sums(0);
    inv_rms(c.side_eps);
#pragma unroll
    for (int i = 0; i < NTW; ++i) y[i] = add_x(y[i], (wave + SNW * i) * 16 + c16);
    row_sums(1);
    inv_rms(c.norm.eps);
#pragma unroll
    for (int i = 0; i < NTW; ++i) {
      const int col = (wave + SNW * i) * 16 + c16;
      if (col >= c.ld) continue;
      const float w = col < c.width ? c.norm.w[col * c.norm.stride] : 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        if (4 * g4 + r >= nr) continue;
        const size_t at = (size_t)(r0 + 4 * g4 + r) * c.ld + col;
        c.x[at] = y[i][r];
        ((T*)c.h)[at] = (T)(y[i][r] * rs[r] * w);
      }
    }
  } else {                                           // a wider row: y is computed twice, x goes through memory (every thread reads what it wrote)
    for (int nt = wave, i = 0; nt < ntiles; nt += SNW, ++i) {
      const f32x4 v = y_tile(i);
#pragma unroll
      for (int r = 0; r < 4; ++r) ss[r] += v[r] * v[r];
    }
    row_sums(0);
    inv_rms(c.side_eps);
    for (int nt = wave, i = 0; nt < ntiles; nt += SNW, ++i) {
      const f32x4 v = add_x(y_tile(i), nt * 16 + c16);
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (4 * g4 + r < nr) c.x[(size_t)(r0 + 4 * g4 + r) * c.ld + nt * 16 + c16] = v[r];
    }
    row_sums(1);
    inv_rms(c.norm.eps);
    for (int nt = wave; nt < ntiles; nt += SNW) {
      const int col = nt * 16 + c16;
      const float w = col < c.width ? c.norm.w[col * c.norm.stride] : 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        if (4 * g4 + r >= nr) continue;
        const size_t at = (size_t)(r0 + 4 * g4 + r) * c.ld + col;
        ((T*)c.h)[at] = (T)(c.x[at] * rs[r] * w);
      }
    }
  }
}

template <typename T>
int side_mfma_at(const SideNormCall& c, hipStream_t st) {
  const int dp = (c.dim + 31) & ~31;
  const int lds = std::max(16 * (c.ld + 8) * 2, SNW * (dp / 16) * 1024);
  auto go = [&](auto k) -> int {
    MI_HIP(hipFuncSetAttribute((const void*)k, hipFuncAttributeMaxDynamicSharedMemorySize, 140 * 1024));
    hipLaunchKernelGGL(k, dim3((c.rows + 15) / 16), dim3(SNW * 64), lds, st, c);
    MI_HIP(hipGetLastError());
    return MI_OK;
  };
  if (c.ld <= 512) return go(side_norm_mfma_kernel<T, 4>);
  if (c.ld <= 1024) return go(side_norm_mfma_kernel<T, 8>);
  if (c.ld <= 2048) return go(side_norm_mfma_kernel<T, 16>);
  return go(side_norm_mfma_kernel<T, 0>);
}

constexpr int SIDE_MFMA_ROWS = 64;      // below: a workgroup per row keeps more CUs busy

template <typename T>
int side_norm_at(const SideNormCall& c, hipStream_t st) {
  if constexpr (sizeof(T) == 2) {
    if (c.proj_p != nullptr && c.rows >= SIDE_MFMA_ROWS) return side_mfma_at<T>(c, st);
  }
  const size_t row_bytes = (2 * (size_t)c.ld + c.dim) * sizeof(float);
  const size_t lds_max = 128 * 1024;
  if (row_bytes > lds_max) return fail(MI_ERR_UNSUPPORTED, "side_norm: row too wide for the LDS");
#define GO(NTV, RBV) do { auto k = side_norm_kernel<T, NTV, RBV>; \
    if (RBV * row_bytes > 65536) MI_HIP(hipFuncSetAttribute((const void*)k, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds_max)); \
    hipLaunchKernelGGL(k, dim3((c.rows + RBV - 1) / RBV), dim3(NTV), RBV * row_bytes, st, c); } while (0)
  if (c.rows >= 1024 && 4 * row_bytes <= lds_max) GO(256, 4);
  else if (c.rows >= 512 && 2 * row_bytes <= lds_max) GO(256, 2);
  else GO(1024, 1);
#undef GO
  MI_HIP(hipGetLastError());
  return MI_OK;
}

// ---- norm of a sublayer's output, residual update, operand of what follows: one workgroup per row ------------------------
template <typename T>
__device__ __forceinline__ f32x4 load4v(const T* p) {
  const float4 v = load4f<T>(p);
  return f32x4{v.x, v.y, v.z, v.w};
}
// NQ: pieces of four columns of the row per thread, held in registers (ld <= 4 NT NQ)
template <typename T, int NT, int NQ, bool ROUTE>
__global__ __launch_bounds__(NT) void post_norm_kernel(PostNormCall c) {
  extern __shared__ __attribute__((aligned(16))) float smem[];      // ROUTE: [ld] the row, [experts (even)] logits, weights | marks, [top] choices
  __shared__ float red[NT / 64];
  const int r = blockIdx.x, tid = threadIdx.x, n4 = c.ld / 4;
  const float inv_n = 1.0f / (float)c.width;
  if (c.clear != nullptr && r == 0)
    for (int i = tid; i < c.n_clear; i += NT) c.clear[i] = 0;
  // the first router rows of this wave (columns below 512 PRE) are on their way while the norm runs
  constexpr int JB = 2, PRE = ROUTE && sizeof(T) == 2 && NQ < 4 ? 4 : 0;
  const int lane = tid & 63, wave = tid >> 6;
  u32x4 wpre[JB][PRE > 0 ? PRE : 1];
  if constexpr (PRE > 0) {
#pragma unroll
    for (int j = 0; j < JB; ++j)
#pragma unroll
      for (int i = 0; i < PRE; ++i)
        wpre[j][i] = *(const u32x4*)((const T*)c.router + (size_t)min(wave * JB + j, c.r.experts - 1) * c.ld + min(lane * 8 + 512 * i, c.ld - 8));
  }
  f32x4 y[NQ], x[NQ];
  float* xg = c.x + (size_t)r * c.ld;
#pragma unroll
  for (int q = 0; q < NQ; ++q) {
    const int i = min(q * NT + tid, n4 - 1);
    x[q] = ((const f32x4*)xg)[i];
    if (c.y != nullptr) y[q] = ((const f32x4*)(c.y + (size_t)r * c.ld))[i];
    else {
      const T* p = (const T*)c.parts + (size_t)r * c.top * c.ld + 4 * i;
      const float* pw = c.part_w + (size_t)r * c.top;
      f32x4 a = {0.f, 0.f, 0.f, 0.f};
      if (c.shared) a = load4v<T>((const T*)c.parts + ((size_t)c.rows * c.top + r) * c.ld + 4 * i);
#pragma unroll 4
      for (int j = 0; j < c.top; ++j) {
        const f32x4 v = load4v<T>(p + (size_t)j * c.ld);
        const float w = pw[j];
#pragma unroll
        for (int i4 = 0; i4 < 4; ++i4) a[i4] = fmaf(w, v[i4], a[i4]);
      }
      y[q] = a;
    }
  }
  // element k = 4 (q NT + tid) + j of the row counts when k < width
  auto each = [&](auto f) {
#pragma unroll
    for (int q = 0; q < NQ; ++q)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int k = 4 * (q * NT + tid) + j;
        if (k < c.width) f(q, j, k);
      }
  };
  // v <- norm of the row: mean taken off for a layer norm, weight w, bias b
  auto normed = [&](f32x4 (&v)[NQ], const PostNormW& n) {
    float mean = 0.f, s[1] = {0.f};
    if (c.kind == MI_NORM_LAYER) {
      each([&](int q, int j, int k) { s[0] += v[q][j]; });
      block_sum<NT, 1>(s, red);
      mean = s[0] * inv_n;
    }
    s[0] = 0.f;
    each([&](int q, int j, int k) { const float d = v[q][j] - mean; s[0] += d * d; });
    block_sum<NT, 1>(s, red);
    const float rs = 1.0f / sqrtf(s[0] * inv_n + c.eps);
    each([&](int q, int j, int k) {
      float e = (v[q][j] - mean) * rs * n.w[(size_t)k * n.stride];
      if (n.b != nullptr) e += n.b[k];
      v[q][j] = e;
    });
  };
  normed(y, c.norm);
  each([&](int q, int j, int k) { x[q][j] += y[q][j]; });
#pragma unroll
  for (int q = 0; q < NQ; ++q) {
    const int i = q * NT + tid;
    if (i >= n4) continue;
    ((f32x4*)xg)[i] = x[q];
  }
  if (c.next.w != nullptr) normed(x, c.next);
  T* h = (T*)c.h + (size_t)r * c.ld;
#pragma unroll
  for (int q = 0; q < NQ; ++q) {
    const int i = q * NT + tid;
    if (i >= n4) continue;
    T o[4] = {from_f32<T>(x[q][0]), from_f32<T>(x[q][1]), from_f32<T>(x[q][2]), from_f32<T>(x[q][3])};
    if constexpr (sizeof(T) == 2) *(uint2*)(h + 4 * i) = __builtin_bit_cast(uint2, o);
    else *(f32x4*)(h + 4 * i) = x[q];
    if constexpr (ROUTE) ((f32x4*)smem)[i] = c.next.w != nullptr ? f32x4{to_f32(o[0]), to_f32(o[1]), to_f32(o[2]), to_f32(o[3])} : x[q];
  }
  if constexpr (ROUTE) {
    float* z = smem + c.ld;
    float* sw = z + ((c.r.experts + 1) & ~1);
    int* sel = (int*)(sw + route_lds_floats(c.r));
    __syncthreads();
    for (int e0 = wave * JB; e0 < c.r.experts; e0 += NT / 64 * JB) {
      float acc[JB] = {0.f, 0.f};
      auto add = [&](int k, const float (&w)[JB][8]) {
        float xv[8];
        load8f<float>(smem + k, xv);
#pragma unroll
        for (int j = 0; j < JB; ++j)
#pragma unroll
          for (int i = 0; i < 8; ++i) acc[j] = fmaf(w[j][i], xv[i], acc[j]);
      };
      int k0 = lane * 8;
      if constexpr (PRE > 0) {
        if (e0 == wave * JB) {
#pragma unroll
          for (int q = 0; q < PRE; ++q, k0 += 512)
            if (k0 < c.ld) {
              float w[JB][8];
#pragma unroll
              for (int j = 0; j < JB; ++j) {
                const T* e = (const T*)&wpre[j][q];
#pragma unroll
                for (int i = 0; i < 8; ++i) w[j][i] = to_f32(e[i]);
              }
              add(k0, w);
            }
        }
      }
#pragma unroll 2
      for (int k = k0; k < c.ld; k += 512) {
        float w[JB][8];
#pragma unroll
        for (int j = 0; j < JB; ++j) load8f<T>((const T*)c.router + (size_t)min(e0 + j, c.r.experts - 1) * c.ld + k, w[j]);
        add(k, w);
      }
#pragma unroll
      for (int j = 0; j < JB; ++j) {
        const float v = wave_sum(acc[j]);
        if (lane == 0 && e0 + j < c.r.experts) z[e0 + j] = c.r.bias != nullptr ? v + c.r.bias[e0 + j] : v;
      }
    }
    __syncthreads();
    if (wave == 0) route_wave(z, c.r, sel, sw, c.ids + (size_t)r * c.r.top, c.wts + (size_t)r * c.r.top);
  }
}

template <typename T>
int post_norm_at(const PostNormCall& c, hipStream_t st) {
  const bool route = c.router != nullptr;
  const size_t lds = !route ? 0 : ((size_t)c.ld + c.r.experts + 1 + route_lds_floats(c.r) + c.r.top) * sizeof(float);
  if (lds > 128 * 1024) return fail(MI_ERR_UNSUPPORTED, "post_norm: row too wide for the LDS");
  auto go = [&](auto k, int nt) -> int {
    if (lds > 65536) MI_HIP(hipFuncSetAttribute((const void*)k, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    hipLaunchKernelGGL(k, dim3(c.rows), dim3(nt), lds, st, c);
    MI_HIP(hipGetLastError());
    return MI_OK;
  };
#define PN(NT, NQ) return route ? go(post_norm_kernel<T, NT, NQ, true>, NT) : go(post_norm_kernel<T, NT, NQ, false>, NT)
  if (c.rows < 256) {                                  // few rows: more threads for each
    if (c.ld <= 4096) PN(1024, 1);
    if (c.ld <= 8192) PN(1024, 2);
    if (c.ld <= 16384) PN(1024, 4);
  }
  if (c.ld <= 1024) PN(256, 1);
  if (c.ld <= 2048) PN(256, 2);
  if (c.ld <= 4096) PN(512, 2);
  if (c.ld <= 8192) PN(1024, 2);
  if (c.ld <= 16384) PN(1024, 4);
#undef PN
  return fail(MI_ERR_UNSUPPORTED, "post_norm: rows of more than 16384 columns");
}

__global__ __launch_bounds__(256) void logit_cap_kernel(float* z, size_t n, float scale, float cap) {
  for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (size_t)gridDim.x * 256) {
    const float v = z[i] * scale;
    z[i] = cap > 0.f ? cap * tanhf(v / cap) : v;
  }
}

__global__ void advance_segments_kernel(SegTables t, int32_t* off, const int32_t* tokens, int32_t* prev) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i >= t.n) return;
  off[t.row[i]] += t.len[i];                         // (distinct rows)
  if (prev != nullptr) prev[t.row[i]] = tokens[t.tok0[i] + t.len[i] - 1];
}

// one workgroup per row; NT threads x 4 NQ columns.  S: number of streams, 0: c.streams of them (at most MAX_STREAMS)
template <typename T, int NT, int NQ, int S>
__global__ __launch_bounds__(NT) void stream_norm_kernel(StreamNormCall c) {
  constexpr int MS = S > 0 ? S : MAX_STREAMS;
  __shared__ float red[NT / 64];
  const int r = blockIdx.x, tid = threadIdx.x, n4 = c.ld / 4, ns = S > 0 ? S : c.streams;
  float* xg = c.x + (size_t)r * ns * c.ld;
  f32x4 u[NQ];
  float ss[1] = {0.f};
#pragma unroll
  for (int q = 0; q < NQ; ++q) {
    const int i = q * NT + tid;
    u[q] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (i >= n4) continue;
    f32x4 x[MS];
#pragma unroll
    for (int s = 0; s < MS; ++s) if (s < ns) x[s] = ((const f32x4*)(xg + (size_t)s * c.ld))[i];
    const f32x4 y = ((const f32x4*)(c.y + (size_t)r * c.ld))[i] * c.mult;
#pragma unroll
    for (int t = 0; t < MS; ++t) {
      if (t >= ns) continue;
      f32x4 v;
      if (c.mix != nullptr) {
        v = y * c.out[t];
#pragma unroll
        for (int s = 0; s < MS; ++s) if (s < ns) v += x[s] * c.mix[s * ns + t];
      } else v = x[t] + y;
      if (c.store) ((f32x4*)(xg + (size_t)t * c.ld))[i] = v;
      u[q] += c.in != nullptr ? v * c.in[t] : v;
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) if (4 * i + j < c.width) ss[0] += u[q][j] * u[q][j];
  }
  block_sum<NT, 1>(ss, red);
  const float rs = 1.0f / sqrtf(ss[0] / (float)c.width + c.norm.eps);
  T* h = (T*)c.h + (size_t)r * c.ld;
#pragma unroll
  for (int q = 0; q < NQ; ++q) {
    const int i = q * NT + tid;
    if (i >= n4) continue;
    T o[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) { const int k = 4 * i + j; o[j] = from_f32<T>(k < c.width ? u[q][j] * rs * c.norm.w[k * c.norm.stride] : 0.f); }
    if constexpr (sizeof(T) == 2) *(uint2*)(h + 4 * i) = __builtin_bit_cast(uint2, o);
    else *(f32x4*)(h + 4 * i) = __builtin_bit_cast(f32x4, o);
  }
}

template <typename T, int S>
int stream_norm_s(const StreamNormCall& c, hipStream_t st) {
#define SN(NT, NQ) do { hipLaunchKernelGGL((stream_norm_kernel<T, NT, NQ, S>), dim3(c.rows), dim3(NT), 0, st, c); MI_HIP(hipGetLastError()); return MI_OK; } while (0)
  if (c.rows < 256) {                                  // few rows: more threads for each
    if (c.ld <= 1024) SN(256, 1);
    if (c.ld <= 2048) SN(512, 1);
    if (c.ld <= 4096) SN(1024, 1);
    if (c.ld <= 8192) SN(1024, 2);
    if (c.ld <= 16384) SN(1024, 4);
  }
  if (c.ld <= 1024) SN(256, 1);
  if (c.ld <= 2048) SN(256, 2);
  if (c.ld <= 4096) SN(512, 2);
  if (c.ld <= 8192) SN(1024, 2);
  if (c.ld <= 16384) SN(1024, 4);
#undef SN
  return fail(MI_ERR_UNSUPPORTED, "stream_norm: rows of more than 16384 columns");
}
template <typename T>
int stream_norm_at(const StreamNormCall& c, hipStream_t st) {
  switch (c.streams) {
    case 0: case 1: return stream_norm_s<T, 1>(c, st);
    case 2: return stream_norm_s<T, 2>(c, st);
    case 3: return stream_norm_s<T, 3>(c, st);
    case 4: return stream_norm_s<T, 4>(c, st);
    default: return stream_norm_s<T, 0>(c, st);
  }
}

__global__ __launch_bounds__(256) void stream_sum_kernel(const float* x, int streams, int rows, int ld, float* out) {
  for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < (size_t)rows * ld; i += (size_t)gridDim.x * 256) {
    const size_t r = i / ld, k = i % ld;
    float v = 0.f;
    for (int s = 0; s < streams; ++s) v += x[(r * streams + s) * ld + k];
    out[i] = v;
  }
}

__global__ __launch_bounds__(256) void rotation_table_kernel(float2* tab, int positions, int half, const double* freq, double gain) {
  for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < (size_t)positions * half; i += (size_t)gridDim.x * 256) {
    const double a = (double)(i / half) * freq[i % half];
    tab[i] = float2{(float)(gain * cos(a)), (float)(gain * sin(a))};
  }
}

template <typename E>
__global__ __launch_bounds__(256) void place_kernel(PlaceCall c) {
  const size_t n = (size_t)c.nb * c.ni * c.nj;
  for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (size_t)gridDim.x * 256) {
    const size_t b = i / ((size_t)c.ni * c.nj), q = i % ((size_t)c.ni * c.nj), ii = q / c.nj, jj = q % c.nj;
    ((E*)c.dst)[b * c.db + ii * c.di + jj * c.dj] = ((const E*)c.src)[b * c.sb + ii * c.si + jj * c.sj];
  }
}

}  // namespace

int launch_embed_pos(const EmbedPosCall& c, hipStream_t st) {
  // few rows: more threads for each
#define GO(TT) do { if (c.t.R < 256) hipLaunchKernelGGL((embed_pos_kernel<TT, 1024>), dim3(c.t.R), dim3(1024), 0, st, c); \
    else hipLaunchKernelGGL((embed_pos_kernel<TT, 256>), dim3(c.t.R), dim3(256), 0, st, c); } while (0)
  switch (c.act) {
    case MI_F32: GO(float); break;
    case MI_BF16: GO(bf16); break;
    case MI_F16: GO(f16); break;
    default: return fail(MI_ERR_INVALID, "embed_pos: bad dtype");
  }
#undef GO
  MI_HIP(hipGetLastError());
  return MI_OK;
}

bool side_mfma_supported(int act, int dim, int ld) { return act != MI_F32 && dim >= 1 && dim <= 128 && ld <= 4096; }

int launch_side_norm(const SideNormCall& c, hipStream_t st) {
  if (c.ld % 8 != 0) return fail(MI_ERR_INVALID, "side_norm: row stride must be a multiple of 8");
  switch (c.act) {
    case MI_F32: return side_norm_at<float>(c, st);
    case MI_BF16: return side_norm_at<bf16>(c, st);
    case MI_F16: return side_norm_at<f16>(c, st);
  }
  return fail(MI_ERR_INVALID, "side_norm: bad dtype");
}

int launch_post_norm(const PostNormCall& c, hipStream_t st) {
  if (c.ld % 8 != 0) return fail(MI_ERR_INVALID, "post_norm: row stride must be a multiple of 8");
  switch (c.act) {
    case MI_F32: return post_norm_at<float>(c, st);
    case MI_BF16: return post_norm_at<bf16>(c, st);
    case MI_F16: return post_norm_at<f16>(c, st);
  }
  return fail(MI_ERR_INVALID, "post_norm: bad dtype");
}

int launch_logit_cap(float* logits, size_t n, float scale, float softcap, hipStream_t st) {
  if (n == 0 || (scale == 1.0f && softcap <= 0.f)) return MI_OK;
  hipLaunchKernelGGL(logit_cap_kernel, dim3((unsigned)std::min<size_t>((n + 255) / 256, 8192)), dim3(256), 0, st, logits, n, scale, softcap);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_advance_segments(const SegTables& t, int32_t* off, const int32_t* tokens, int32_t* prev, hipStream_t st) {
  hipLaunchKernelGGL(advance_segments_kernel, dim3((t.n + 255) / 256), dim3(256), 0, st, t, off, tokens, prev);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_stream_norm(const StreamNormCall& c, hipStream_t st) {
  if (c.ld % 8 != 0 || c.streams < 0 || c.streams > MAX_STREAMS || c.norm.w == nullptr || (c.mix == nullptr) != (c.out == nullptr) ||
      (c.streams > 1 && c.mix == nullptr))
    return fail(MI_ERR_INVALID, "stream_norm: bad call");
  switch (c.act) {
    case MI_F32: return stream_norm_at<float>(c, st);
    case MI_BF16: return stream_norm_at<bf16>(c, st);
    case MI_F16: return stream_norm_at<f16>(c, st);
  }
  return fail(MI_ERR_INVALID, "stream_norm: bad dtype");
}

int launch_stream_sum(const float* x, int streams, int rows, int ld, float* out, hipStream_t st) {
  hipLaunchKernelGGL(stream_sum_kernel, dim3((unsigned)std::min<size_t>(((size_t)rows * ld + 255) / 256, 4096)), dim3(256), 0, st, x, streams, rows, ld, out);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_rotation_table(float2* tab, int positions, int pairs, const double* freq, double gain, hipStream_t st) {
  const size_t n = (size_t)positions * pairs;
  hipLaunchKernelGGL(rotation_table_kernel, dim3((unsigned)std::min<size_t>((n + 255) / 256, 8192)), dim3(256), 0, st, tab, positions, pairs, freq, gain);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

int launch_place(const PlaceCall& c, hipStream_t st) {
  const size_t n = (size_t)c.nb * c.ni * c.nj;
  if (n == 0) return MI_OK;
  const dim3 grid((unsigned)std::min<size_t>((n + 255) / 256, 4096)), block(256);
  if (c.es == 4) hipLaunchKernelGGL(place_kernel<uint32_t>, grid, block, 0, st, c);
  else hipLaunchKernelGGL(place_kernel<uint16_t>, grid, block, 0, st, c);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

}  // namespace mi
