// lightning.hip -- linear attention with a fixed decay per head (layer-list models).  q, k and v have been through silu (the epilogue of
// their projection); per head  S <- decay S + k v^T,  o = S^T q  with S in float32;  out = rms(o of all heads) * norm * sigmoid(gate).
//
// State per cache row: S transposed, [value column][key channel].  A row whose length is 0 starts from zero: nothing has to be cleared
// when a row is used again.
//
// One-token segments: ONE launch, a workgroup per (segment, head, strip of value columns): S read once and written once, the outputs
// summed over the key channels on the way; the last workgroup of a token to arrive makes its norm and gate.
// Longer segments of bfloat16 models, in chunks (the decay of a chunk does not depend on the tokens, so only a sum of small matrices is
// sequential; n = tokens of the chunk, i and j count in it):
//   light_chunk  a workgroup per (chunk, head): K^T diag(decay^(n-1-j)) V
//   light_carry  a thread per four elements of S: the states in front of the chunks, left in place of those as 16-bit pairs hi + lo
//   light_out    a workgroup per (64 queries, head): decay^(i+1) (Q S) + (Q K^T o decay^(i-j), j <= i) V
//   light_norm   a workgroup per token: norm over all heads, gate
// Operands that carry a decay or the state enter the matrix products as 16-bit pairs hi + lo, so they keep 32-bit accuracy.
// Float32 and float16 (whose range a state may leave), and head sizes above 128: light_scan, token by token.
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

template <typename T>
__device__ __forceinline__ f32x4 mfma16(u32x4 a, u32x4 b, f32x4 c) {
  if constexpr (std::is_same<T, bf16>::value)
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
  else
    return __builtin_amdgcn_mfma_f32_16x16x32_f16(__builtin_bit_cast(f16x8, a), __builtin_bit_cast(f16x8, b), c, 0, 0, 0);
}

// two float32 values as hi + lo pairs of 16-bit values
template <typename T>
__device__ __forceinline__ void split2(float a, float b, uint32_t& hi, uint32_t& lo) {
  typedef float f32x2 __attribute__((ext_vector_type(2)));
  typedef T tx2 __attribute__((ext_vector_type(2)));
  const tx2 h = __builtin_convertvector((f32x2{a, b}), tx2);
  const f32x2 back = __builtin_convertvector(h, f32x2);
  hi = __builtin_bit_cast(uint32_t, h);
  lo = __builtin_bit_cast(uint32_t, __builtin_convertvector((f32x2{a - back[0], b - back[1]}), tx2));
}

// elements [k, k + 8) of a head of n, zeros beyond
template <typename T>
__device__ __forceinline__ u32x4 head8(const T* p, int k, int n) {
  if (n % 8 == 0 && ((uintptr_t)p & 15) == 0) {
    if (k < n) return *(const u32x4*)(p + k);
    return u32x4{0, 0, 0, 0};
  }
  T v[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) v[i] = k + i < n ? p[k + i] : from_f32<T>(0.f);
  return __builtin_bit_cast(u32x4, v);
}

// decay^n (n = 0 gives 1 also for a decay of zero)
__device__ __forceinline__ float decay_pow(float log2_decay, int n) { return __builtin_amdgcn_exp2f(log2_decay * (float)n); }

// sum over aligned groups of L lanes (a power of two)
template <int L>
__device__ __forceinline__ float lanes_sum(float v) {
  if constexpr (L >= 16) {
    v = row16_sum(v);
    if constexpr (L >= 32) v += __shfl_xor(v, 16, 64);
    if constexpr (L >= 64) v += __shfl_xor(v, 32, 64);
    return v;
  } else {
#pragma unroll
    for (int x = 1; x < L; x *= 2) v += __shfl_xor(v, x, 64);
    return v;
  }
}

// norm over all heads and gate of token r by NT threads; o(k): output k of the token.  NQ > 0: four consecutive outputs per thread and
// round, NQ rounds, in registers (n a multiple of four); 0: any n
template <typename T, int NT, int NQ, typename F>
__device__ __forceinline__ void norm_and_gate(const LightCall& c, int r, float* red, F o) {
  const int n = c.H * c.e;
  if constexpr (NQ > 0) {
    const T* gate = (const T*)c.proj + (size_t)r * c.ldp + c.o_g;
    f32x4 v[NQ], w[NQ];
    float4 z[NQ];
    float ss[1] = {0.f};
#pragma unroll
    for (int q = 0; q < NQ; ++q) {                     // (one round trip)
      const int k = min(4 * (q * NT + (int)threadIdx.x), n - 4);
      v[q] = o(k);
      w[q] = *(const f32x4*)(c.norm + k);
      z[q] = load4f<T>(gate + k);
    }
#pragma unroll
    for (int q = 0; q < NQ; ++q) {
      if (4 * (q * NT + (int)threadIdx.x) >= n) continue;
#pragma unroll
      for (int j = 0; j < 4; ++j) ss[0] += v[q][j] * v[q][j];
    }
    block_sum<NT, 1>(ss, red);
    const float rs = 1.0f / sqrtf(ss[0] / (float)n + c.eps);
#pragma unroll
    for (int q = 0; q < NQ; ++q) {
      const int k = 4 * (q * NT + (int)threadIdx.x);
      if (k >= n) continue;
      const float g[4] = {z[q].x, z[q].y, z[q].z, z[q].w};
      T out[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) out[j] = from_f32<T>(v[q][j] * rs * w[q][j] * sigmoid_f(g[j]));
      T* dst = (T*)c.cat + (size_t)r * c.ldc + k;
      if constexpr (sizeof(T) == 2) *(uint2*)dst = __builtin_bit_cast(uint2, out);
      else *(f32x4*)dst = f32x4{(float)out[0], (float)out[1], (float)out[2], (float)out[3]};
    }
    return;
  }
  float ss[1] = {0.f};
  for (int k = threadIdx.x; k < n; k += NT) { const float v = o(k)[0]; ss[0] += v * v; }
  block_sum<NT, 1>(ss, red);
  const float rs = 1.0f / sqrtf(ss[0] / (float)n + c.eps);
  const T* gate = (const T*)c.proj + (size_t)r * c.ldp + c.o_g;
  T* cat = (T*)c.cat + (size_t)r * c.ldc;
  for (int k = threadIdx.x; k < n; k += NT) cat[k] = from_f32<T>(o(k)[0] * rs * c.norm[k] * sigmoid_f(to_f32(gate[k])));
}

// ---- one-token segments --------------------------------------------------------------------------------------------------
// grid (nd, H, strips of DE value columns), 4 waves.  L lanes share a column, NV pieces of four key channels each (4 L NV >= d).
// NQ: of norm_and_gate.  The new state is stored behind the ticket, so nobody waits for it.
constexpr int DE = 32;
template <typename T, int L, int NV, int NQ>
__global__ __launch_bounds__(256) void light_decode_kernel(LightCall c) {
  constexpr int CPW = 64 / L, STEP = 4 * CPW, NI = (DE + STEP - 1) / STEP;      // columns per wave and step, steps
  __shared__ float red[4];
  __shared__ int last_sh;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, sl = lane % L, cw = wave * CPW + lane / L;
  const int seg = c.t.dec[blockIdx.x], r = c.t.tok0[seg], row = c.t.row[seg], pos = c.t.off[row], h = blockIdx.y, e0 = blockIdx.z * DE;
  const T* pr = (const T*)c.proj + (size_t)r * c.ldp;
  float* S = c.state + ((size_t)row * c.H + h) * (size_t)c.e * c.sd;
  f32x4 s[NI][NV];
#pragma unroll
  for (int i = 0; i < NI; ++i)
#pragma unroll
    for (int v = 0; v < NV; ++v) {
      const int col = min(e0 + i * STEP + cw, c.e - 1), k = 4 * (sl + v * L);
      s[i][v] = pos > 0 ? *(const f32x4*)(S + (size_t)col * c.sd + min(k, c.sd - 4)) : f32x4{0.f, 0.f, 0.f, 0.f};
    }
  float q[NV][4], kk[NV][4];
#pragma unroll
  for (int v = 0; v < NV; ++v)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int k = 4 * (sl + v * L) + j, kc = min(k, c.d - 1);
      const float qv = to_f32(pr[c.o_q + h * c.d + kc]), kv = to_f32(pr[c.o_k + h * c.d + kc]);
      q[v][j] = k < c.d ? qv : 0.f;
      kk[v][j] = k < c.d ? kv : 0.f;
    }
  const float g = c.decay[h];
  float* o = c.o + (size_t)r * c.ldo + h * c.e;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int in = i * STEP + cw, col = e0 + in;
    const bool on = in < DE && col < c.e;
    const float vv = to_f32(pr[c.o_v + h * c.e + min(col, c.e - 1)]);
    float a = 0.f;
#pragma unroll
    for (int v = 0; v < NV; ++v) {
      const int k = 4 * (sl + v * L);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        s[i][v][j] = fmaf(kk[v][j], vv, g * s[i][v][j]);
        a = fmaf(s[i][v][j], q[v][j], a);
      }
    }
    a = lanes_sum<L>(a);
    if (on && sl == 0) __hip_atomic_store(&o[col], a, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  }
  // the last workgroup of the token to arrive (nobody waits): outputs are at agent scope, the ticket follows them
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();
  if (tid == 0) {
    const int ticket = __hip_atomic_fetch_add(&c.tickets[blockIdx.x], 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    last_sh = ticket == (int)(gridDim.y * gridDim.z) - 1;
    if (last_sh) __hip_atomic_store(&c.tickets[blockIdx.x], 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  }
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int in = i * STEP + cw, col = e0 + in;
#pragma unroll
    for (int v = 0; v < NV; ++v) {
      const int k = 4 * (sl + v * L);
      if (in < DE && col < c.e && k < c.sd) *(f32x4*)(S + (size_t)col * c.sd + k) = s[i][v];
    }
  }
  __syncthreads();
  if (!last_sh) return;
  const float* all = c.o + (size_t)r * c.ldo;
  norm_and_gate<T, 256, NQ>(c, r, red, [&](int k) {
    f32x4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < (NQ > 0 ? 4 : 1); ++j) v[j] = __hip_atomic_load(&all[k + j], __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    return v;
  });
}

// ---- token by token ------------------------------------------------------------------------------------------------------
// grid (ceil(e / 16), H, segments of two tokens and more), 16 lanes per value column, DPL key channels per lane
template <typename T, int DPL>
__global__ __launch_bounds__(256) void light_scan_kernel(LightCall c) {
  const int seg = c.t.chunk[blockIdx.z], h = blockIdx.y, row = c.t.row[seg], r0 = c.t.tok0[seg], n = c.t.len[seg], off = c.t.off[row];
  const int sl = threadIdx.x & 15, col = blockIdx.x * 16 + (threadIdx.x >> 4), colc = min(col, c.e - 1);
  float* S = c.state + (((size_t)row * c.H + h) * c.e + colc) * (size_t)c.sd;
  const float g = c.decay[h];
  float s[DPL];
#pragma unroll
  for (int i = 0; i < DPL; ++i) s[i] = off > 0 && sl + 16 * i < c.d ? S[sl + 16 * i] : 0.f;
  for (int t = 0; t < n; ++t) {
    const T* pr = (const T*)c.proj + (size_t)(r0 + t) * c.ldp;
    const float v = to_f32(pr[c.o_v + h * c.e + colc]);
    float a = 0.f;
#pragma unroll
    for (int i = 0; i < DPL; ++i) {
      const int k = sl + 16 * i;
      if (k < c.d) {
        s[i] = fmaf(to_f32(pr[c.o_k + h * c.d + k]), v, g * s[i]);
        a = fmaf(s[i], to_f32(pr[c.o_q + h * c.d + k]), a);
      }
    }
    a = row16_sum(a);
    if (sl == 0 && col < c.e) c.o[(size_t)(r0 + t) * c.ldo + h * c.e + col] = a;
  }
  if (col >= c.e) return;
#pragma unroll
  for (int i = 0; i < DPL; ++i)
    if (sl + 16 * i < c.sd) S[sl + 16 * i] = s[i];
}

template <typename T, int NQ>
__global__ __launch_bounds__(256) void light_norm_kernel(LightCall c) {
  __shared__ float red[4];
  const int r = blockIdx.x;
  if (c.t.len[c.t.tok_seg[r]] < 2) return;
  const float* o = c.o + (size_t)r * c.ldo;
  norm_and_gate<T, 256, NQ>(c, r, red, [&](int k) {
    if constexpr (NQ > 0) return *(const f32x4*)(o + k);
    else return f32x4{o[k], 0.f, 0.f, 0.f};
  });
}

// ---- chunks --------------------------------------------------------------------------------------------------------------
// LDS images that are read transposed: [32 tokens][16 columns] tiles of 32-byte rows, tile (half of the block, columns / 16)
template <int W>
__device__ __forceinline__ size_t timg(int token, int piece) {       // byte of the 16-byte piece (eight columns) of a token
  return (size_t)((token >> 5) * (W / 16) + (piece >> 1)) * 1024 + ((token & 31) ^ ((piece >> 1) & 7)) * 32 + (piece & 1) * 16;
}
// operand of columns 16 ct .. (this lane: column c16) over the 32 tokens of half hf: slots 4 g4 .. and 16 + 4 g4 ..
template <int W>
__device__ __forceinline__ u32x4 tread(const unsigned char* img, int hf, int ct, int c16, int g4) {
  const unsigned char* a = img + (size_t)(hf * (W / 16) + ct) * 1024 + ((4 * g4 + (c16 >> 2)) ^ (ct & 7)) * 32 + (c16 & 3) * 8;
  const s16x4 v0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)a);
  const s16x4 v1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)(a + 16 * 32));
  const uint32_t* w0 = (const uint32_t*)&v0;
  const uint32_t* w1 = (const uint32_t*)&v1;
  return u32x4{w0[0], w0[1], w1[0], w1[1]};
}

// grid (H, chunks), 4 waves: wave (wd, we) has every WD-th 16-channel tile of the keys and every WE-th 16-column tile of the values
template <typename T, int DP, int EP>
__global__ __launch_bounds__(256, 3) void light_chunk_kernel(LightCall c) {
  constexpr int KB = 64, WD = DP >= 64 ? 4 : 2, WE = 4 / WD, ND = DP / 16 / WD, NE = EP / 16 / WE;
  constexpr int NKP = (KB * DP / 8 + 255) / 256, NVP = (KB * EP / 8 + 255) / 256;          // 16-byte pieces per thread
  __shared__ __attribute__((aligned(16))) unsigned char khi[KB * DP * 2], klo[KB * DP * 2], vim[KB * EP * 2];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c16 = lane & 15, g4 = lane >> 4, wd = wave % WD, we = wave / WD;
  const int h = blockIdx.x, seg = c.ctile[2 * blockIdx.y], t0 = c.ctile[2 * blockIdx.y + 1];
  const int r0 = c.t.tok0[seg] + t0, n = min(c.chunk, c.t.len[seg] - t0);
  const float l2 = c.log2_decay[h];
  const T* kp = (const T*)c.proj + (size_t)r0 * c.ldp + c.o_k + h * c.d;
  const T* vp = (const T*)c.proj + (size_t)r0 * c.ldp + c.o_v + h * c.e;
  u32x4 kreg[NKP], vreg[NVP];
  auto load = [&](int b) {
#pragma unroll
    for (int i = 0; i < NKP; ++i) {
      const int p = i * 256 + tid, t = b + p / (DP / 8);
      kreg[i] = head8<T>(kp + (size_t)min(t, n - 1) * c.ldp, 8 * (p % (DP / 8)), c.d);
    }
#pragma unroll
    for (int i = 0; i < NVP; ++i) {
      const int p = i * 256 + tid, t = b + p / (EP / 8);
      vreg[i] = head8<T>(vp + (size_t)min(t, n - 1) * c.ldp, 8 * (p % (EP / 8)), c.e);
    }
  };
  f32x4 acc[ND][NE];
#pragma unroll
  for (int i = 0; i < ND; ++i)
#pragma unroll
    for (int j = 0; j < NE; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  load(0);
  for (int b = 0; b < n; b += KB) {
    if (b > 0) __syncthreads();                        // (the images have been read)
#pragma unroll
    for (int i = 0; i < NKP; ++i) {
      const int p = i * 256 + tid, t = p / (DP / 8);
      if (t >= KB) continue;
      const float f = b + t < n ? decay_pow(l2, n - 1 - b - t) : 0.f;       // (tokens beyond the end add nothing)
      const T* x = (const T*)&kreg[i];
      uint32_t hi[4], lo[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) split2<T>(to_f32(x[2 * j]) * f, to_f32(x[2 * j + 1]) * f, hi[j], lo[j]);
      *(u32x4*)(khi + timg<DP>(t, p % (DP / 8))) = u32x4{hi[0], hi[1], hi[2], hi[3]};
      *(u32x4*)(klo + timg<DP>(t, p % (DP / 8))) = u32x4{lo[0], lo[1], lo[2], lo[3]};
    }
#pragma unroll
    for (int i = 0; i < NVP; ++i) {
      const int p = i * 256 + tid, t = p / (EP / 8);
      if (t < KB) *(u32x4*)(vim + timg<EP>(t, p % (EP / 8))) = vreg[i];
    }
    load(min(b + KB, n - 1));
    __syncthreads();
#pragma unroll
    for (int hf = 0; hf < KB / 32; ++hf) {
      u32x4 a[ND][2];
#pragma unroll
      for (int i = 0; i < ND; ++i) {
        a[i][0] = tread<DP>(khi, hf, wd + WD * i, c16, g4);
        a[i][1] = tread<DP>(klo, hf, wd + WD * i, c16, g4);
      }
#pragma unroll
      for (int j = 0; j < NE; ++j) {
        const u32x4 v = tread<EP>(vim, hf, we + WE * j, c16, g4);
#pragma unroll
        for (int i = 0; i < ND; ++i) {
          acc[i][j] = mfma16<T>(a[i][0], v, acc[i][j]);
          acc[i][j] = mfma16<T>(a[i][1], v, acc[i][j]);
        }
      }
    }
  }
  float* out = c.ws + ((size_t)blockIdx.y * c.H + h) * DP * EP;
#pragma unroll
  for (int i = 0; i < ND; ++i)
#pragma unroll
    for (int j = 0; j < NE; ++j) *(f32x4*)(out + (size_t)(16 * (we + WE * j) + c16) * DP + 16 * (wd + WD * i) + 4 * g4) = acc[i][j];
}

// grid (H DP EP / 1024, segments of two tokens and more): the states in front of the chunks, as [4 hi][4 lo] per four elements
template <typename T, int DP, int EP>
__global__ __launch_bounds__(256) void light_carry_kernel(LightCall c) {
  constexpr int PER = DP * EP / 4, U = 8;
  const int i = blockIdx.x * 256 + threadIdx.x, h = i / PER, at = i % PER * 4, col = at / DP, k = at % DP;
  const int seg = c.t.chunk[blockIdx.y], row = c.t.row[seg], len = c.t.len[seg], off = c.t.off[row], nc = (len + c.chunk - 1) / c.chunk;
  const bool in = col < c.e && k < c.sd;
  float* S = c.state + (((size_t)row * c.H + h) * c.e + min(col, c.e - 1)) * (size_t)c.sd + min(k, c.sd - 4);
  f32x4 s = off > 0 && in ? *(const f32x4*)S : f32x4{0.f, 0.f, 0.f, 0.f};
  float* ws = c.ws + ((size_t)c.cbase[seg] * c.H + h) * DP * EP + at;
  const size_t ld = (size_t)c.H * DP * EP;
  const float whole = decay_pow(c.log2_decay[h], c.chunk), rest = decay_pow(c.log2_decay[h], len - (nc - 1) * c.chunk);
  for (int b = 0; b < nc; b += U) {
    f32x4 v[U];
#pragma unroll
    for (int u = 0; u < U; ++u) v[u] = *(const f32x4*)(ws + (size_t)min(b + u, nc - 1) * ld);
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (b + u >= nc) break;
      uint32_t hi[2], lo[2];
      split2<T>(s[0], s[1], hi[0], lo[0]);
      split2<T>(s[2], s[3], hi[1], lo[1]);
      *(u32x4*)(ws + (size_t)(b + u) * ld) = u32x4{hi[0], hi[1], lo[0], lo[1]};
      s = s * (b + u == nc - 1 ? rest : whole) + v[u];
    }
  }
  if (in) *(f32x4*)S = s;
}

// grid (H, chunks x chunk / LIGHT_QT), 4 waves of 16 queries each.  The products are laid out as in the attention kernels:
// rows = keys / state columns / output columns, columns = queries.
template <typename T, int DP, int EP>
__global__ __launch_bounds__(256, 4) void light_out_kernel(LightCall c) {
  constexpr int KB = 64, KK = DP / 32, ET = EP / 16, SB = EP < 64 ? EP : 64;               // SB: state columns staged at a time
  constexpr int NKP = (KB * DP / 8 + 255) / 256, NVP = (KB * EP / 8 + 255) / 256, NSP = (SB * DP / 8 + 255) / 256;
  constexpr int AIMG = KB * DP * 2, BIMG = KB * (EP > DP ? EP : DP) * 2;
  __shared__ __attribute__((aligned(16))) unsigned char ia[AIMG], ib[BIMG];      // state hi, lo; then keys, values
  const int per = c.chunk / LIGHT_QT, ck = blockIdx.y / per, t0 = blockIdx.y % per * LIGHT_QT;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c16 = lane & 15, g4 = lane >> 4;
  const int h = blockIdx.x, seg = c.ctile[2 * ck], s0 = c.ctile[2 * ck + 1], n = min(c.chunk, c.t.len[seg] - s0);
  if (t0 >= n) return;
  const int r0 = c.t.tok0[seg] + s0, q = t0 + wave * 16 + c16;         // this lane's query, in the chunk
  const bool zero = s0 == 0 && c.t.off[c.t.row[seg]] == 0;             // (no state in front of the chunk)
  const float l2 = c.log2_decay[h];
  const T* base = (const T*)c.proj + (size_t)r0 * c.ldp;
  const T* kp = base + c.o_k + h * c.d;
  const T* vp = base + c.o_v + h * c.e;
  u32x4 qf[KK];
#pragma unroll
  for (int kk = 0; kk < KK; ++kk) qf[kk] = head8<T>(base + (size_t)min(q, n - 1) * c.ldp + c.o_q + h * c.d, 32 * kk + 8 * g4, c.d);
  // rows that are left operands: [16-row tile][kk][g][row ^ (4 kk + g)] x 16 bytes
  auto at = [&](int row, int piece) { return (size_t)(((row >> 4) * KK * 4 + piece) * 16 + ((row ^ piece) & 15)) * 16; };
  auto frag = [&](const unsigned char* img, int tile, int kk) {
    return *(const u32x4*)(img + (size_t)((tile * KK * 4 + 4 * kk + g4) * 16 + (c16 ^ ((4 * kk + g4) & 15))) * 16);
  };
  u32x4 kreg[NKP], vreg[NVP];
  auto load = [&](int b) {
#pragma unroll
    for (int i = 0; i < NKP; ++i) {
      const int p = i * 256 + tid;
      kreg[i] = head8<T>(kp + (size_t)min(b + p / (DP / 8), n - 1) * c.ldp, 8 * (p % (DP / 8)), c.d);
    }
#pragma unroll
    for (int i = 0; i < NVP; ++i) {
      const int p = i * 256 + tid;
      vreg[i] = head8<T>(vp + (size_t)min(b + p / (EP / 8), n - 1) * c.ldp, 8 * (p % (EP / 8)), c.e);
    }
  };
  f32x4 acc[ET];
#pragma unroll
  for (int i = 0; i < ET; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  if (!zero) {
    const float* S = c.ws + ((size_t)ck * c.H + h) * DP * EP;
#pragma unroll
    for (int sb = 0; sb < EP; sb += SB) {
      u32x4 x[NSP][2];
#pragma unroll
      for (int i = 0; i < NSP; ++i) {
        const int p = min(i * 256 + tid, SB * DP / 8 - 1);
        const float* s = S + (size_t)(sb + p / (DP / 8)) * DP + 8 * (p % (DP / 8));
        x[i][0] = *(const u32x4*)s;
        x[i][1] = *(const u32x4*)(s + 4);
      }
      if (sb > 0) __syncthreads();
#pragma unroll
      for (int i = 0; i < NSP; ++i) {
        const int p = i * 256 + tid;
        if (p >= SB * DP / 8) continue;
        *(u32x4*)(ia + at(p / (DP / 8), p % (DP / 8))) = u32x4{x[i][0][0], x[i][0][1], x[i][1][0], x[i][1][1]};
        *(u32x4*)(ib + at(p / (DP / 8), p % (DP / 8))) = u32x4{x[i][0][2], x[i][0][3], x[i][1][2], x[i][1][3]};
      }
      __syncthreads();
#pragma unroll
      for (int e = 0; e < SB / 16; ++e)
#pragma unroll
        for (int kk = 0; kk < KK; ++kk) {
          acc[sb / 16 + e] = mfma16<T>(frag(ia, e, kk), qf[kk], acc[sb / 16 + e]);
          acc[sb / 16 + e] = mfma16<T>(frag(ib, e, kk), qf[kk], acc[sb / 16 + e]);
        }
    }
    const float f = decay_pow(l2, q + 1);
#pragma unroll
    for (int i = 0; i < ET; ++i) acc[i] *= f;
    __syncthreads();
  }
  load(0);
  for (int b = 0; b <= t0; b += KB) {                  // key blocks up to the diagonal's
    if (b > 0) __syncthreads();
#pragma unroll
    for (int i = 0; i < NKP; ++i) {
      const int p = i * 256 + tid;
      if (p < KB * DP / 8) *(u32x4*)(ia + at(p / (DP / 8), p % (DP / 8))) = kreg[i];
    }
#pragma unroll
    for (int i = 0; i < NVP; ++i) {
      const int p = i * 256 + tid;
      if (p < KB * EP / 8) *(u32x4*)(ib + timg<EP>(p / (EP / 8), p % (EP / 8))) = vreg[i];
    }
    load(min(b + KB, t0));
    __syncthreads();
#pragma unroll
    for (int hf = 0; hf < 2; ++hf) {
      uint32_t ph[4], pl[4];
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        f32x4 sc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kk = 0; kk < KK; ++kk) sc = mfma16<T>(frag(ia, 2 * hf + t, kk), qf[kk], sc);
        const int dist = q - (b + 32 * hf + 16 * t + 4 * g4);           // to the lane's first key
#pragma unroll
        for (int r = 0; r < 4; ++r) sc[r] = dist >= r ? sc[r] * decay_pow(l2, dist - r) : 0.f;
        split2<T>(sc[0], sc[1], ph[2 * t], pl[2 * t]);
        split2<T>(sc[2], sc[3], ph[2 * t + 1], pl[2 * t + 1]);
      }
      const u32x4 pf = {ph[0], ph[1], ph[2], ph[3]}, pg = {pl[0], pl[1], pl[2], pl[3]};
#pragma unroll
      for (int e = 0; e < ET; ++e) {
        const u32x4 v = tread<EP>(ib, hf, e, c16, g4);
        acc[e] = mfma16<T>(v, pf, acc[e]);
        acc[e] = mfma16<T>(v, pg, acc[e]);
      }
    }
  }
  if (q >= n) return;
  float* o = c.o + (size_t)(r0 + q) * c.ldo + h * c.e;
#pragma unroll
  for (int e = 0; e < ET; ++e) {
    const int k = 16 * e + 4 * g4;
    if (c.e % 4 == 0) { if (k < c.e) *(f32x4*)(o + k) = acc[e]; }
    else {
#pragma unroll
      for (int r = 0; r < 4; ++r) if (k + r < c.e) o[k + r] = acc[e][r];
    }
  }
}

int pad(int n) { return n <= 32 ? 32 : (n <= 64 ? 64 : 128); }

template <typename T, int DP, int EP>
int chunks_de(const LightCall& c, hipStream_t st) {
  hipLaunchKernelGGL((light_chunk_kernel<T, DP, EP>), dim3(c.H, c.nct), dim3(256), 0, st, c);
  MI_HIP(hipGetLastError());
  hipLaunchKernelGGL((light_carry_kernel<T, DP, EP>), dim3(c.H * DP * EP / 1024, c.t.nc), dim3(256), 0, st, c);
  MI_HIP(hipGetLastError());
  hipLaunchKernelGGL((light_out_kernel<T, DP, EP>), dim3(c.H, c.nct * (c.chunk / LIGHT_QT)), dim3(256), 0, st, c);
  MI_HIP(hipGetLastError());
  return MI_OK;
}

template <typename T>
int chunks_at(const LightCall& c, hipStream_t st) {
  if constexpr (std::is_same<T, bf16>::value) {
    if (c.chunk < LIGHT_QT || c.chunk % LIGHT_QT != 0 || c.nct < 1 || c.ldo % 4 != 0) return fail(MI_ERR_INVALID, "lightning: bad chunks");
    const int dp = pad(c.d), ep = pad(c.e);
#define V(DP, EP) if (dp == DP && ep == EP) return chunks_de<T, DP, EP>(c, st);
    V(32, 32) V(32, 64) V(32, 128) V(64, 32) V(64, 64) V(64, 128) V(128, 32) V(128, 64) V(128, 128)
#undef V
  }
  return fail(MI_ERR_UNSUPPORTED, "lightning: chunks of bfloat16 models with head sizes up to 128 only");
}

template <typename T>
int scan_at(const LightCall& c, hipStream_t st) {
  const dim3 grid((c.e + 15) / 16, c.H, c.t.nc), block(256);
  const int dpl = (c.d + 15) / 16;
#define GO(D) hipLaunchKernelGGL((light_scan_kernel<T, D>), grid, block, 0, st, c)
  if (dpl <= 2) GO(2); else if (dpl <= 4) GO(4); else if (dpl <= 8) GO(8); else if (dpl <= 16) GO(16); else GO(32);
#undef GO
  MI_HIP(hipGetLastError());
  return MI_OK;
}

template <typename T>
int light_at(const LightCall& c, hipStream_t st) {
  // rounds of four outputs per thread of the norm, 0: element by element
  const int n = c.H * c.e, nq = n % 4 == 0 && n <= 8 * 1024 && c.ldo % 4 == 0 && c.ldc % 4 == 0 ? (n + 1023) / 1024 : 0;
  if (c.t.nd > 0) {
    const dim3 grid(c.t.nd, c.H, (c.e + DE - 1) / DE), block(256);
#define GO(L, NV) do { if (nq == 0) hipLaunchKernelGGL((light_decode_kernel<T, L, NV, 0>), grid, block, 0, st, c); \
    else if (nq <= 2) hipLaunchKernelGGL((light_decode_kernel<T, L, NV, 2>), grid, block, 0, st, c); \
    else hipLaunchKernelGGL((light_decode_kernel<T, L, NV, 8>), grid, block, 0, st, c); } while (0)
    if (c.d <= 16) GO(4, 1); else if (c.d <= 32) GO(8, 1); else if (c.d <= 64) GO(16, 1); else if (c.d <= 128) GO(32, 1);
    else if (c.d <= 256) GO(64, 1); else GO(64, 2);
#undef GO
    MI_HIP(hipGetLastError());
  }
  if (c.t.nc > 0) {
    if (c.ws != nullptr) MI_TRY(chunks_at<T>(c, st));
    else MI_TRY(scan_at<T>(c, st));
#define GO(NQ) hipLaunchKernelGGL((light_norm_kernel<T, NQ>), dim3(c.t.R), dim3(256), 0, st, c)
    if (nq == 0) GO(0); else if (nq <= 1) GO(1); else if (nq <= 2) GO(2); else if (nq <= 4) GO(4); else GO(8);
#undef GO
    MI_HIP(hipGetLastError());
  }
  return MI_OK;
}

}  // namespace

bool light_supported(int d, int e) { return d >= 1 && d <= 512 && e >= 1 && e <= 4096; }
size_t light_ws_floats(int act, int H, int d, int e) {
  return act == MI_BF16 && d <= 128 && e <= 128 ? (size_t)H * pad(d) * pad(e) : 0;
}

int launch_lightning(const LightCall& c, hipStream_t st) {
  if (!light_supported(c.d, c.e) || c.sd % 4 != 0 || c.sd < c.d || c.sd > c.d + 3) return fail(MI_ERR_UNSUPPORTED, "lightning: head sizes not supported");
  if (c.t.nd > 0 && c.tickets == nullptr) return fail(MI_ERR_INVALID, "lightning: no tickets");
  switch (c.act) {
    case MI_F32: return light_at<float>(c, st);
    case MI_BF16: return light_at<bf16>(c, st);
    case MI_F16: return light_at<f16>(c, st);
  }
  return fail(MI_ERR_INVALID, "lightning: bad dtype");
}

}  // namespace mi
