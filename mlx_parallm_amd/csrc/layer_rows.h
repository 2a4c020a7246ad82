// layer_rows.h -- device helpers of the row-wise kernels of layer-list models (one workgroup per token row).
#pragma once
#include "layer_kernels.h"

namespace mi {
namespace rows {

// sum over a workgroup of NT threads; every thread gets the result.  `red` holds NT / 64 floats per value.
template <int NT, int NV>
__device__ __forceinline__ void block_sum(float (&v)[NV], float* red) {
  constexpr int NW = NT / 64;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
#pragma unroll
  for (int i = 0; i < NV; ++i) v[i] = wave_sum(v[i]);
  __syncthreads();                                   // (red may still be read from a previous sum)
  if (lane == 0) {
#pragma unroll
    for (int i = 0; i < NV; ++i) red[wave * NV + i] = v[i];
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    float s = 0.f;
#pragma unroll
    for (int w = 0; w < NW; ++w) s += red[w * NV + i];
    v[i] = s;
  }
}

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_f(float z) { return z * sigmoid_f(z); }
__device__ __forceinline__ float softplus_f(float z) { return z > 20.f ? z : log1pf(expf(z)); }
__device__ __forceinline__ float gelu_tanh_f(float z) {
  return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

// position of token r, and its place
struct TokenAt { int seg, row, t, pos, off; };
__device__ __forceinline__ TokenAt token_at(const SegTables& s, int r) {
  TokenAt a;
  a.seg = s.tok_seg[r];
  a.row = s.row[a.seg];
  a.t = r - s.tok0[a.seg];
  a.off = s.off[a.row];
  a.pos = a.off + a.t;
  return a;
}

// Rotated coordinate j of `dims`: its partner, the pair's number, and the sign of  partner * sine  (j's own value times the cosine is
// added).  Partners are dims / 2 apart, or neighbours (pairs).
struct RotAt { int partner, f; float sign; };
__device__ __forceinline__ RotAt rot_at(int j, int dims, int pairs) {
  if (pairs) return RotAt{j ^ 1, j >> 1, (j & 1) ? 1.f : -1.f};
  const int half = dims >> 1;
  return j < half ? RotAt{j + half, j, -1.f} : RotAt{j - half, j - half, 1.f};
}

// eight / four consecutive elements as float32 (16- / 8-byte aligned)
template <typename T>
__device__ __forceinline__ void load8f(const T* p, float (&o)[8]) {
  if constexpr (sizeof(T) == 4) {
    const float4 a = *(const float4*)p, b = *(const float4*)(p + 4);
    o[0] = a.x; o[1] = a.y; o[2] = a.z; o[3] = a.w; o[4] = b.x; o[5] = b.y; o[6] = b.z; o[7] = b.w;
  } else {
    const uint4 v = *(const uint4*)p;
    const T* e = (const T*)&v;
#pragma unroll
    for (int i = 0; i < 8; ++i) o[i] = (float)e[i];
  }
}
template <typename T>
__device__ __forceinline__ void store8f(T* p, const float (&v)[8]) {
  T o[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) o[i] = from_f32<T>(v[i]);
  if constexpr (sizeof(T) == 4) { *(uint4*)p = *(const uint4*)o; *(uint4*)(p + 4) = *(const uint4*)(o + 4); }
  else *(uint4*)p = *(const uint4*)o;
}
template <typename T>
__device__ __forceinline__ float4 load4f(const T* p) {
  if constexpr (sizeof(T) == 4) return *(const float4*)p;
  else {
    const uint2 v = *(const uint2*)p;
    const T* e = (const T*)&v;
    return float4{(float)e[0], (float)e[1], (float)e[2], (float)e[3]};
  }
}

// PolyNorm of one row by one workgroup: out = a N(z) + b N(z^2) + c N(z^3) + e.  z and out 16-byte aligned.
template <typename T, int NT>
__device__ __forceinline__ void polynorm_row(const PolyNormArgs& f, const T* z, T* out, float* red) {
  float s[3] = {0.f, 0.f, 0.f};
  const int full = f.ff & ~7;
  auto add = [&](float v) { const float v2 = v * v; s[0] += v2; s[1] += v2 * v2; s[2] += v2 * v2 * v2; };
  for (int i = threadIdx.x * 8; i < full; i += NT * 8) {
    float v[8];
    load8f<T>(z + i, v);
#pragma unroll
    for (int j = 0; j < 8; ++j) add(v[j]);
  }
  const int tail = full + (int)threadIdx.x;
  if (tail < f.ff) add(to_f32(z[tail]));
  block_sum<NT, 3>(s, red);
  const float n = (float)f.ff;
  const float ca = f.coef[0] / sqrtf(s[0] / n + f.eps), cb = f.coef[1] / sqrtf(s[1] / n + f.eps),
              cc = f.coef[2] / sqrtf(s[2] / n + f.eps), ce = f.coef[3];
  for (int i = threadIdx.x * 8; i < full; i += NT * 8) {
    float v[8];
    load8f<T>(z + i, v);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = ((cc * v[j] + cb) * v[j] + ca) * v[j] + ce;
    store8f<T>(out + i, v);
  }
  if (tail < f.ff) { const float v = to_f32(z[tail]); out[tail] = from_f32<T>(((cc * v + cb) * v + ca) * v + ce); }
}

// Routing of one token by one wave: z [E] logits in LDS -> the `top` experts with the largest softmax scores among the `keep`
// groups with the largest best score, in falling order, and their weights (scores over their sum).  `sel`: [top] in LDS, `sw`:
// route_lds_floats() floats of LDS, 8-byte aligned.  Ranks by counting, the others' values broadcast from their lanes: no expert or
// group is taken twice, ties go to the lower number.
__device__ __forceinline__ float lane_value(float v, int lane) {
  return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), lane));
}
// how many of the n values v(i) come before (mine, me) in falling order
template <typename F>
__device__ __forceinline__ int rank_of(float mine, int me, int n, F v) {
  const int lane = threadIdx.x & 63;
  int rank = 0;
  for (int b = 0; b < n; b += 64) {
    const float vb = v(min(b + lane, n - 1));
    const int k = min(64, n - b);
#pragma unroll 8
    for (int o = 0; o < k; ++o) {
      const float x = lane_value(vb, o);
      rank += x > mine || (x == mine && b + o < me) ? 1 : 0;
    }
  }
  return rank;
}
__device__ __forceinline__ void route_wave(const float* z, const RouteArgs& r, int* sel, float* sw, int32_t* ids, float* wts) {
  const int lane = threadIdx.x & 63, E = r.experts, gs = E / r.groups;
  unsigned long long* marks = (unsigned long long*)sw;                 // a bit per kept group
  float* gbest = sw + 2 * ((r.groups + 63) / 64);                      // [groups] best logit of a group
  float* wsel = gbest + r.groups;                                      // [top]
  for (int j = lane; j < r.top; j += 64) { sel[j] = j; wsel[j] = 0.f; }
  float zm = -INFINITY;
  for (int e = lane; e < E; e += 64) zm = fmaxf(zm, z[e]);
  zm = wave_max(zm);
  float tot = 0.f;
  for (int e = lane; e < E; e += 64) tot += expf(z[e] - zm);
  tot = wave_sum(tot);
  const bool grouped = r.keep < r.groups;
  if (grouped) {
    for (int g = lane; g < r.groups; g += 64) {
      float best = -INFINITY;
#pragma unroll 8
      for (int i = 0; i < gs; ++i) best = fmaxf(best, z[g * gs + i]);
      gbest[g] = best;
    }
    for (int g0 = 0; g0 < r.groups; g0 += 64) {
      const int g = min(g0 + lane, r.groups - 1);
      const int ahead = rank_of(gbest[g], g, r.groups, [&](int o) { return gbest[o]; });
      const unsigned long long m = __builtin_amdgcn_ballot_w64(g0 + lane < r.groups && ahead < r.keep);
      if (lane == 0) marks[g0 >> 6] = m;
    }
  }
  auto kept = [&](int e) {                             // the expert's logit, -inf outside the kept groups
    const float v = z[e];
    if (!grouped) return v;
    const int g = e / gs;
    return marks[g >> 6] >> (g & 63) & 1 ? v : -INFINITY;
  };
  float chosen = 0.f;
  for (int e0 = 0; e0 < E; e0 += 64) {
    const int e = min(e0 + lane, E - 1);
    const float ze = kept(e);
    const int rank = rank_of(ze, e, E, kept);
    if (e0 + lane < E && ze > -INFINITY && rank < r.top) {
      const float s = expf(ze - zm) / tot;
      sel[rank] = e; wsel[rank] = s;
      chosen += s;
    }
  }
  chosen = wave_sum(chosen) + 1e-20f;
  for (int j = lane; j < r.top; j += 64) { ids[j] = sel[j]; wts[j] = wsel[j] / chosen; }
}
// floats of LDS behind `sw`, an even number: marks, groups, weights
__host__ __device__ constexpr int route_lds_floats(const RouteArgs& r) { return (2 * ((r.groups + 63) / 64) + r.groups + r.top + 1) & ~1; }

}  // namespace rows
}  // namespace mi
