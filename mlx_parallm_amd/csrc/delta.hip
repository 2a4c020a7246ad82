// delta.hip -- gated delta rule with short convolutions (layer-list models).
//
//   q, k, v  = silu(short causal convolution of the projections);  q, k unit vectors per head, q scaled
//   beta     = sigmoid(b),  g = exp(-exp(A_log) softplus(a + dt_bias))                      per value head
//   S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q                            S: [d][e] float32
//   out      = rms(o) * w * silu(gate)       (or sigmoid)
// The second form (channel) has a decay g_c per value head and key channel: row c of S is multiplied by g_c.
//
// State per cache row: S, and the last inputs of the convolutions in a ring (the input of position p lies in slot p mod taps:
// a step reads the slots of p-1 .. p-taps+1 and writes the one of p, so the workgroups that share a q/k head may read while
// one of them writes).  A row whose length is 0 starts from zero: nothing has to be cleared when a row is used again.
//
// One-token segments: ONE launch, a workgroup per (segment, value head).  With a = (g S)^T k and b = (g S)^T q from a single
// pass over S, u = beta (v - a) and o = b + (k . q) u, so S is read once and written once.
// Longer segments, whole chunks of 64 tokens at a time (float32 matrix-core products throughout; float64 sums of the log decays):
//   delta_conv   convolutions and activations, all tokens and channels in parallel
//   delta_chunk  a workgroup per (chunk, value head).  With G the running sum of log g inside the chunk, A_ij = beta_i e^(G_i - G_j)
//                k_i . k_j (j < i), T = (I + A)^-1:  W = T diag(beta e^G) K,  U = T diag(beta) V,  P_ij = e^(G_i - G_j) q_i . k_j (j <= i)
//   delta_carry  the chunks of a segment in order, a workgroup per 16 columns of S:
//                X = U - W S,  O = diag(e^G) Q S + P X,  S <- e^(G_last) S + K^T diag(e^(G_last - G)) X
// With a decay per channel the factors belong to elements of Q and K instead of rows: delta_chunk_channel makes
//                A_ij = beta_i sum_c k_ic k_jc D_ijc,  P_ij = sum_c q_ic k_jc D_ijc,  D_ijc = product of g_c over the tokens j + 1 .. i
// without ever dividing by a decay: between blocks of 16 tokens D is (start of i's block .. i) x (blocks between) x (j + 1 .. end of j's
// block), each at most one, so those tiles are matrix products of scaled rows; inside a block D is a running product.
// Short portions, and sizes the chunk kernels do not take: delta_prep (convolutions, norms, gates, all tokens in parallel) ->
// delta_scan (token by token; columns of S are independent, so a wave owns four columns and keeps them in registers, 16 lanes
// per column).  Both end in delta_out.
#include <algorithm>
#include <type_traits>

#include "layer_rows.h"

namespace mi {

namespace {

using namespace rows;

// one channel of a short convolution at token r (segment position t, absolute position pos), before the activation
template <typename T>
__device__ __forceinline__ float conv_at(const T* proj, size_t ldp, int col, int r, int t, int pos, const T* ring, int C, int chan,
                                         const float* taps, int K) {
  float y = taps[K - 1] * to_f32(proj[(size_t)r * ldp + col]);
  for (int j = 1; j < K; ++j) {
    if (pos - j < 0) break;                          // zeros before the start
    const float x = j <= t ? to_f32(proj[(size_t)(r - j) * ldp + col]) : to_f32(ring[(size_t)((pos - j) % K) * C + chan]);
    y = fmaf(taps[K - 1 - j], x, y);
  }
  return y;
}

struct Chan { int col; const float* taps; };
// channel ch of [q: Gd | k: Gd | v: He] -> its column in the projections and its taps
__device__ __forceinline__ Chan channel(const DeltaCall& c, int ch) {
  const int gd = c.G * c.d;
  if (ch < gd) return {c.o_q + ch, c.conv_q + (size_t)ch * c.taps};
  if (ch < 2 * gd) return {c.o_k + ch - gd, c.conv_k + (size_t)(ch - gd) * c.taps};
  return {c.o_v + ch - 2 * gd, c.conv_v + (size_t)(ch - 2 * gd) * c.taps};
}

// i: the head, or (channel) head * d + channel
__device__ __forceinline__ float decay_of(const DeltaCall& c, int h, int i, float a) {
  return expf(-expf(c.A_log[h]) * softplus_f(a + c.dt_bias[i]));
}
template <typename T>
__device__ __forceinline__ float out_gate(const DeltaCall& c, int r, int i) {
  const float z = to_f32(((const T*)c.gp)[(size_t)r * c.ldgp + c.o_g + i]);
  return c.gate_act == MI_GATE_SIGMOID ? sigmoid_f(z) : silu_f(z);
}

// The outer low-rank maps of one token and value head by a workgroup of NT threads: decays[d] and gates[e] from the inner
// projections in the token's row `pr`.  P neighbouring threads share an output.
template <typename T, int NT>
__device__ __forceinline__ void low_rank_rows(const DeltaCall& c, const T* pr, int h, float* decays, float* gates) {
  const int tid = threadIdx.x, n = c.d + c.e;
  int P = 1;
  while (P < 8 && 2 * P * n <= NT) P *= 2;
  for (int o0 = 0; o0 < n; o0 += NT / P) {
    const int o = o0 + tid / P, p = tid % P;
    const bool isa = o < c.d, on = o < n;
    const T* w = isa ? (const T*)c.low_a + (size_t)(h * c.d + o) * c.ld_a : (const T*)c.low_g + (size_t)(h * c.e + min(o, n - 1) - c.d) * c.ld_gt;
    const T* x = pr + (isa ? c.in_a : c.in_g);
    const int len = isa ? c.ld_a : c.ld_gt;
    float s = 0.f;
#pragma unroll 8
    for (int k = 8 * p; k < len; k += 8 * P) {
      float a[8], b[8];
      load8f<T>(w + k, a);
      load8f<T>(x + k, b);
#pragma unroll
      for (int i = 0; i < 8; ++i) s = fmaf(a[i], b[i], s);
    }
    for (int m = 1; m < P; m *= 2) s += __shfl_xor(s, m, 64);
    if (on && p == 0) {
      if (isa) decays[o] = decay_of(c, h, h * c.d + o, s);
      else gates[o - c.d] = c.gate_act == MI_GATE_SIGMOID ? sigmoid_f(s) : silu_f(s);
    }
  }
}

template <int VEC> struct Vec;
template <> struct Vec<1> { float v[1]; };
template <> struct alignas(16) Vec<4> { float v[4]; };

// grid (one-token segments, H + (ff ? 1 : 0)).  MAXR > 0: the thread's rows of S stay in registers between the two passes.
// CHAN: a decay per channel.
constexpr int DNT = 512;
template <typename T, int VEC, int MAXR, bool CHAN>
__global__ __launch_bounds__(DNT) void delta_decode_kernel(DeltaCall c) {
  __shared__ float red[DNT / 64 * 3];
  __shared__ Vec<VEC> part[2][DNT];
  __shared__ float ks[512], qs[512], gs[CHAN ? 512 : 1], og[CHAN ? DNT * VEC : 1];
  __shared__ float vs[DNT * VEC];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int seg = c.t.dec[blockIdx.x], r = c.t.tok0[seg], row = c.t.row[seg], pos = c.t.off[row];
  const T* proj = (const T*)c.proj;
  const T* pr = proj + (size_t)r * c.ldp;
  T* cat = (T*)c.cat + (size_t)r * c.ldc;
  const int h = blockIdx.y;
  if (h == c.H) {                                    // the feed-forward activation rides in this launch
    polynorm_row<T, DNT>(c.ff, pr + c.ff.in_off, cat + c.ff.out_off, red);
    return;
  }
  const int d = c.d, e = c.e, K = c.taps, hg = c.H / c.G, gq = h / hg, C = 2 * c.G * d + c.H * e;
  T* ring = (T*)c.ring + (size_t)row * K * C;
  float* S = c.state + ((size_t)row * c.H + h) * (size_t)d * e;
  const int ncol = e / VEC, slices = DNT / ncol, col = tid % ncol, sl = tid / ncol;
  const bool on = sl < slices;

  // S first: the longest latency
  Vec<VEC> s[MAXR > 0 ? MAXR : 1];
  if constexpr (MAXR > 0) {
    if (pos > 0 && on) {
#pragma unroll
      for (int i = 0; i < MAXR; ++i) {
        const int dr = min(sl + i * slices, d - 1);
        s[i] = *(const Vec<VEC>*)(S + (size_t)dr * e + col * VEC);
      }
    } else {
#pragma unroll
      for (int i = 0; i < MAXR; ++i)
#pragma unroll
        for (int j = 0; j < VEC; ++j) s[i].v[j] = 0.f;
    }
  }
  for (int i = tid; i < 2 * d + e; i += DNT) {
    const int ch = i < d ? gq * d + i : (i < 2 * d ? c.G * d + gq * d + (i - d) : 2 * c.G * d + h * e + (i - 2 * d));
    const Chan cn = channel(c, ch);
    const float y = silu_f(conv_at<T>(proj, c.ldp, cn.col, r, 0, pos, ring, C, ch, cn.taps, K));
    if (i < d) qs[i] = y; else if (i < 2 * d) ks[i - d] = y; else vs[i - 2 * d] = y;
    if (i >= 2 * d || h % hg == 0) ring[(size_t)(pos % K) * C + ch] = pr[cn.col];
  }
  const T* ar = (const T*)c.ap + (size_t)r * c.ldap + c.o_a;
  if constexpr (CHAN) {
    if (c.low_a != nullptr) low_rank_rows<T, DNT>(c, pr, h, gs, og);
    else {
      for (int i = tid; i < d; i += DNT) gs[i] = decay_of(c, h, h * d + i, to_f32(ar[h * d + i]));
      for (int i = tid; i < e; i += DNT) og[i] = out_gate<T>(c, r, h * e + i);
    }
  }
  __syncthreads();
  float n3[3] = {0.f, 0.f, 0.f};
  for (int i = tid; i < d; i += DNT) { n3[0] += qs[i] * qs[i]; n3[1] += ks[i] * ks[i]; n3[2] += qs[i] * ks[i]; }
  block_sum<DNT, 3>(n3, red);
  const float iq = c.scale / sqrtf(n3[0] + c.unit_eps), ik = 1.0f / sqrtf(n3[1] + c.unit_eps);
  const float kq = n3[2] * iq * ik;
  const float beta = sigmoid_f(to_f32(pr[c.o_b + h]));
  float g = 1.f;
  if constexpr (!CHAN) g = decay_of(c, h, h, to_f32(ar[h]));
  auto row_decay = [&](int dr) { if constexpr (CHAN) return gs[dr]; else return g; };      // of row dr of S
  auto in_row = [&](const float* x, int dr) { if constexpr (CHAN) return x[dr] * gs[dr]; else return x[dr]; };   // (one decay: applied to the sums)

  Vec<VEC> pa, pb;
#pragma unroll
  for (int j = 0; j < VEC; ++j) { pa.v[j] = 0.f; pb.v[j] = 0.f; }
  if (on) {
    if constexpr (MAXR > 0) {
#pragma unroll
      for (int i = 0; i < MAXR; ++i) {
        const int dr = sl + i * slices;
        const float kk = dr < d ? in_row(ks, dr) : 0.f, qq = dr < d ? in_row(qs, dr) : 0.f;
#pragma unroll
        for (int j = 0; j < VEC; ++j) { pa.v[j] = fmaf(s[i].v[j], kk, pa.v[j]); pb.v[j] = fmaf(s[i].v[j], qq, pb.v[j]); }
      }
    } else if (pos > 0) {
      for (int dr = sl; dr < d; dr += slices) {
        const Vec<VEC> x = *(const Vec<VEC>*)(S + (size_t)dr * e + col * VEC);
#pragma unroll
        for (int j = 0; j < VEC; ++j) { pa.v[j] = fmaf(x.v[j], in_row(ks, dr), pa.v[j]); pb.v[j] = fmaf(x.v[j], in_row(qs, dr), pb.v[j]); }
      }
    }
    part[0][tid] = pa; part[1][tid] = pb;
  }
  __syncthreads();
  // u and o of every column (slices summed in order; each thread needs u of its own columns only)
  Vec<VEC> u, o;
  float so[1] = {0.f};
  if (on) {
    Vec<VEC> a, b;
#pragma unroll
    for (int j = 0; j < VEC; ++j) { a.v[j] = 0.f; b.v[j] = 0.f; }
    for (int w = 0; w < slices; ++w) {
      const Vec<VEC> x = part[0][w * ncol + col], y = part[1][w * ncol + col];
#pragma unroll
      for (int j = 0; j < VEC; ++j) { a.v[j] += x.v[j]; b.v[j] += y.v[j]; }
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      u.v[j] = beta * (vs[col * VEC + j] - g * ik * a.v[j]);
      o.v[j] = fmaf(kq, u.v[j], g * iq * b.v[j]);
      if (sl == 0) so[0] += o.v[j] * o.v[j];
    }
    if constexpr (MAXR > 0) {
#pragma unroll
      for (int i = 0; i < MAXR; ++i) {
        const int dr = sl + i * slices;
        if (dr < d) {
          const float kk = ks[dr] * ik, gr = row_decay(dr);
          Vec<VEC> x;
#pragma unroll
          for (int j = 0; j < VEC; ++j) x.v[j] = fmaf(kk, u.v[j], gr * s[i].v[j]);
          *(Vec<VEC>*)(S + (size_t)dr * e + col * VEC) = x;
        }
      }
    } else {
      for (int dr = sl; dr < d; dr += slices) {
        Vec<VEC>* p = (Vec<VEC>*)(S + (size_t)dr * e + col * VEC);
        Vec<VEC> x;
#pragma unroll
        for (int j = 0; j < VEC; ++j) x.v[j] = 0.f;
        if (pos > 0) x = *p;
#pragma unroll
        for (int j = 0; j < VEC; ++j) x.v[j] = fmaf(ks[dr] * ik, u.v[j], row_decay(dr) * x.v[j]);
        *p = x;
      }
    }
  }
  block_sum<DNT, 1>(so, red);
  if (on && sl == 0) {
    const float rs = 1.0f / sqrtf(so[0] / (float)e + c.eps);
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      const int k = col * VEC + j;
      float gate;
      if constexpr (CHAN) gate = og[k]; else gate = out_gate<T>(c, r, h * e + k);
      cat[h * e + k] = from_f32<T>(o.v[j] * rs * c.head_norm[k] * gate);
    }
  }
  (void)lane; (void)wave;
}

// ---- longer segments -----------------------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void delta_prep_kernel(DeltaCall c) {
  const int r = blockIdx.x;
  const TokenAt at = token_at(c.t, r);
  if (c.t.len[at.seg] < 2) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int gd = c.G * c.d, C = 2 * gd + c.H * c.e, K = c.taps;
  const T* proj = (const T*)c.proj;
  const T* ring = (const T*)c.ring + (size_t)at.row * K * C;
  float* out = c.scan + (size_t)r * c.lds;
  const T* pr = proj + (size_t)r * c.ldp;
  const T* ar = (const T*)c.ap + (size_t)r * c.ldap + c.o_a;
  const int hg = c.H / c.G;
  // q and k: a wave per q/k head, which also leaves the gates of its value heads
  for (int hh = wave; hh < c.G; hh += 4) {
    float sq = 0.f, sk = 0.f, qk = 0.f;
    for (int i = lane; i < c.d; i += 64) {
      const int ch = hh * c.d + i;
      const Chan a = channel(c, ch), b = channel(c, gd + ch);
      const float q = silu_f(conv_at<T>(proj, c.ldp, a.col, r, at.t, at.pos, ring, C, ch, a.taps, K));
      const float k = silu_f(conv_at<T>(proj, c.ldp, b.col, r, at.t, at.pos, ring, C, gd + ch, b.taps, K));
      sq += q * q; sk += k * k; qk += q * k;
      out[ch] = q; out[gd + ch] = k;
    }
    const float iq = c.scale / sqrtf(wave_sum(sq) + c.unit_eps), ik = 1.0f / sqrtf(wave_sum(sk) + c.unit_eps);
    qk = wave_sum(qk) * iq * ik;
    for (int i = lane; i < c.d; i += 64) { out[hh * c.d + i] *= iq; out[gd + hh * c.d + i] *= ik; }   // (each lane rescales what it wrote)
    for (int j = lane; j < hg; j += 64) {
      const int h = hh * hg + j;
      float* ga = c.gate + (size_t)r * c.ldg + 4 * h;
      *(float4*)ga = float4{c.channel ? 1.f : decay_of(c, h, h, to_f32(ar[h])), sigmoid_f(to_f32(pr[c.o_b + h])), qk, 0.f};
    }
  }
  for (int i = tid; i < c.H * c.e; i += 256) {
    const Chan cn = channel(c, 2 * gd + i);
    out[2 * gd + i] = silu_f(conv_at<T>(proj, c.ldp, cn.col, r, at.t, at.pos, ring, C, 2 * gd + i, cn.taps, K));
  }
  if (c.channel)
    for (int i = tid; i < c.H * c.d; i += 256) out[C + i] = decay_of(c, i / c.d, i, to_f32(ar[i]));
}

// the last inputs of a segment's convolutions into the ring (whoever reads it in this call ran in an earlier launch);
// the workgroup of the 16 value columns starting at 16 cg of head h, 256 threads
template <typename T>
__device__ __forceinline__ void put_ring(const DeltaCall& c, int h, int gq, int cg, int row, int off, int r0, int n) {
  const int tid = threadIdx.x, gd = c.G * c.d, C = 2 * gd + c.H * c.e, K = c.taps, hg = c.H / c.G, m = min(K, n);
  T* ring = (T*)c.ring + (size_t)row * K * C;
  const T* proj = (const T*)c.proj;
  auto put = [&](int ch) {
    const int cl = channel(c, ch).col;
    for (int j = 0; j < m; ++j) {
      const int t = n - 1 - j;
      ring[(size_t)((off + t) % K) * C + ch] = proj[(size_t)(r0 + t) * c.ldp + cl];
    }
  };
  if (tid < 16 && cg * 16 + tid < c.e) put(2 * gd + h * c.e + cg * 16 + tid);
  if (cg == 0 && h % hg == 0)
    for (int i = tid; i < 2 * c.d; i += 256) put(i < c.d ? gq * c.d + i : gd + gq * c.d + (i - c.d));
}

// grid (ceil(e / 16), H, chunk segments), 4 waves of 4 columns; DPL state rows per lane (16 lanes x DPL >= d).
// The operands of TC tokens at a time are staged in LDS (two buffers; the next ones travel in registers during the current
// ones' arithmetic): q and k of the head, v of the workgroup's 16 columns, decay, step size and k . q.  Per token, with
// a = S^T k and b = S^T q of the state BEFORE the token:  u = beta (v - g a),  o = g b + (k . q) u,  S <- g S + k u^T.
// CHAN: the head's decays are staged beside q and k, and S is multiplied by them before the two products.
template <typename T, int DPL, bool CHAN>
__global__ __launch_bounds__(256) void delta_scan_kernel(DeltaCall c) {
  constexpr int DP = 16 * DPL;                        // padded state rows
  constexpr int TC = DPL <= 12 || (DPL <= 16 && !CHAN) ? 16 : 8, NR = CHAN ? 3 : 2;
  constexpr int NQK = (TC * NR * DP + 255) / 256;     // staged q / k (/ decay) floats per thread
  __shared__ float qk[2][TC][NR][DP];
  __shared__ float vb[2][TC][16];
  __shared__ float ga[2][TC][4];
  __shared__ float ob[TC][16];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int seg = c.t.chunk[blockIdx.z], h = blockIdx.y;
  const int row = c.t.row[seg], r0 = c.t.tok0[seg], n = c.t.len[seg], off = c.t.off[row];
  const int d = c.d, e = c.e, gd = c.G * d, gq = h / (c.H / c.G);
  const int sl = lane & 15, wc = wave * 4 + (lane >> 4), col = blockIdx.x * 16 + wc;
  const bool cv = col < e;
  const int colc = min(col, e - 1), d0 = sl * DPL;
  float* S = c.state + ((size_t)row * c.H + h) * (size_t)d * e;
  float s[DPL];
#pragma unroll
  for (int i = 0; i < DPL; ++i) s[i] = (off > 0 && d0 + i < d) ? S[(size_t)(d0 + i) * e + colc] : 0.f;

  const float* base = c.scan + (size_t)r0 * c.lds;
  const float* gbase = c.gate + (size_t)r0 * c.ldg + 4 * h;
  float rqk[NQK], rv, rg;
  const int vt = tid >> 4, vc = tid & 15, gt = (tid >> 2) % TC, gi = tid & 3;
  // rows beyond d are staged as zeros; tokens beyond n repeat the last one and are never run
  auto load = [&](int t0) {
#pragma unroll
    for (int i = 0; i < NQK; ++i) {
      const int x = i * 256 + tid, t = min(t0 + x / (NR * DP), n - 1), w = x / DP % NR, dd = x % DP;
      const float v = base[(size_t)t * c.lds + (w < 2 ? w * gd + gq * d : 2 * gd + c.H * e + h * d) + min(dd, d - 1)];
      rqk[i] = dd < d ? v : 0.f;
    }
    rv = base[(size_t)min(t0 + min(vt, TC - 1), n - 1) * c.lds + 2 * gd + h * e + min((int)blockIdx.x * 16 + vc, e - 1)];
    rg = gbase[(size_t)min(t0 + gt, n - 1) * c.ldg + gi];
  };
  auto store = [&](int buf) {
#pragma unroll
    for (int i = 0; i < NQK; ++i) {
      const int x = i * 256 + tid;
      if (x < TC * NR * DP) (&qk[buf][0][0][0])[x] = rqk[i];
    }
    if (vt < TC) vb[buf][vt][vc] = rv;
    if (tid < 4 * TC) ga[buf][gt][gi] = rg;
  };
  load(0);
  store(0);
  __syncthreads();
  for (int t0 = 0, buf = 0; t0 < n; t0 += TC, buf ^= 1) {
    const bool more = t0 + TC < n;
    if (more) load(t0 + TC);
    const int m = min(TC, n - t0);
    for (int t = 0; t < m; ++t) {
      const float* kp = &qk[buf][t][1][d0];
      const float* qp = &qk[buf][t][0][d0];
      const float g = ga[buf][t][0], beta = ga[buf][t][1], kq = ga[buf][t][2], v = vb[buf][t][wc];
      float k[DPL], q[DPL];
#pragma unroll
      for (int i = 0; i < DPL; ++i) { k[i] = kp[i]; q[i] = qp[i]; }
      if constexpr (CHAN) {
#pragma unroll
        for (int i = 0; i < DPL; ++i) s[i] *= qk[buf][t][NR - 1][d0 + i];
      }
      float a[2] = {0.f, 0.f}, b[2] = {0.f, 0.f};
#pragma unroll
      for (int i = 0; i < DPL; ++i) { a[i & 1] = fmaf(s[i], k[i], a[i & 1]); b[i & 1] = fmaf(s[i], q[i], b[i & 1]); }
      const float as = row16_sum(a[0] + a[1]), bs = row16_sum(b[0] + b[1]);
      const float u = beta * (v - g * as);
#pragma unroll
      for (int i = 0; i < DPL; ++i) s[i] = fmaf(s[i], g, k[i] * u);
      if (sl == 0) ob[t][wc] = fmaf(kq, u, g * bs);
    }
    __syncthreads();                                  // every wave is done with buf and ob is complete
    if (more) store(buf ^ 1);
    if (vt < m && blockIdx.x * 16 + vc < e) c.scan[(size_t)(r0 + t0 + vt) * c.lds + 2 * gd + h * e + blockIdx.x * 16 + vc] = ob[vt][vc];
    __syncthreads();
  }
  if (cv) {
#pragma unroll
    for (int i = 0; i < DPL; ++i)
      if (d0 + i < d) S[(size_t)(d0 + i) * e + col] = s[i];
  }
  put_ring<T>(c, h, gq, blockIdx.x, row, off, r0, n);
}

// ---- whole chunks ---------------------------------------------------------------------------------------------------
typedef float f32x4 __attribute__((ext_vector_type(4)));
constexpr int CH = DELTA_CHUNK;                       // 64 = four 16-row tiles
constexpr int TW = 16;                                // tokens per thread of the convolution kernel

// grid (ceil(channels / 1024), chunks, CH / TW): four neighbouring channels per thread, TW tokens with the taps in registers
template <typename T, int K>
__global__ __launch_bounds__(256) void delta_conv_kernel(DeltaCall c) {
  const int gd = c.G * c.d, C = 2 * gd + c.H * c.e, ch = (blockIdx.x * 256 + threadIdx.x) * 4;
  const int seg = c.t.ctile[2 * blockIdx.y], t0 = c.t.ctile[2 * blockIdx.y + 1] + blockIdx.z * TW;
  const int row = c.t.row[seg], r0 = c.t.tok0[seg], len = c.t.len[seg], off = c.t.off[row];
  if (ch >= C || t0 >= len) return;
  const Chan cn = channel(c, ch);                     // (q, k and v start at multiples of four)
  const T* proj = (const T*)c.proj + cn.col;
  const T* ring = (const T*)c.ring + (size_t)row * K * C + ch;
  float w[4][K];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < K; ++j) w[i][j] = cn.taps[i * K + j];
  float4 x[K - 1 + TW];
#pragma unroll
  for (int j = 1; j < K; ++j) {                       // inputs in front of the first token: this call's, the ring's, zeros
    const int t = t0 - j;
    float4 v = {0.f, 0.f, 0.f, 0.f};
    if (t >= 0) v = load4f<T>(proj + (size_t)(r0 + t) * c.ldp);
    else if (off + t >= 0) v = load4f<T>(ring + (size_t)((off + t) % K) * C);
    x[K - 1 - j] = v;
  }
#pragma unroll
  for (int i = 0; i < TW; ++i) x[K - 1 + i] = load4f<T>(proj + (size_t)(r0 + min(t0 + i, len - 1)) * c.ldp);
#pragma unroll
  for (int i = 0; i < TW; ++i) {
    float y[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < K; ++j) {
      y[0] = fmaf(w[0][j], x[i + j].x, y[0]); y[1] = fmaf(w[1][j], x[i + j].y, y[1]);
      y[2] = fmaf(w[2][j], x[i + j].z, y[2]); y[3] = fmaf(w[3][j], x[i + j].w, y[3]);
    }
    if (t0 + i < len)
      *(float4*)(c.scan + (size_t)(r0 + t0 + i) * c.lds + ch) = float4{silu_f(y[0]), silu_f(y[1]), silu_f(y[2]), silu_f(y[3])};
  }
}

__device__ __forceinline__ f32x4 mfma4(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
// four k steps: lane (c16, g4) holds elements 4 g4 .. 4 g4 + 3 of a 16-element slice of its row / column
__device__ __forceinline__ f32x4 mfma_slice(f32x4 a, f32x4 b, f32x4 c) {
#pragma unroll
  for (int j = 0; j < 4; ++j) c = mfma4(a[j], b[j], c);
  return c;
}

// grid (chunks, H), 4 waves.  DP: head size padded to 32, 64 or 128.
template <typename T, int DP>
__global__ __launch_bounds__(256, 2) void delta_chunk_kernel(DeltaCall c) {
  constexpr int LK = DP + 4, LA = CH + 4, NS = DP / 16;
  extern __shared__ __attribute__((aligned(16))) float csm[];
  float* ks = csm;                                    // [CH][LK] unit keys
  float* am = ks + CH * LK;                           // [CH][LA] A below the diagonal; block (i, j) of T lies at block (j, i)
  __shared__ double G[CH];
  __shared__ float be[CH], bg[CH], iq[CH];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c16 = lane & 15, g4 = lane >> 4;
  const int h = blockIdx.y, seg = c.t.ctile[2 * blockIdx.x], t0 = c.t.ctile[2 * blockIdx.x + 1];
  const int r0 = c.t.tok0[seg] + t0, n = min(CH, c.t.len[seg] - t0);
  const int d = c.d, e = c.e, gd = c.G * d, gq = h / (c.H / c.G);
  const float* qb = c.scan + (size_t)r0 * c.lds + gq * d;
  const float* kb = qb + gd;
  float* vb = c.scan + (size_t)r0 * c.lds + 2 * gd + (size_t)h * e;

  // keys and their norms, the queries' norms: four threads per token
  {
    const int t = tid >> 2, p = tid & 3;
    float sk = 0.f, sq = 0.f;
    f32x4 kv[DP / 16];
#pragma unroll
    for (int i = 0; i < DP / 16; ++i) {
      const int k = 16 * i + 4 * p;
      kv[i] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (t < n && k < d) {
        kv[i] = *(const f32x4*)(kb + (size_t)t * c.lds + k);
        const f32x4 q = *(const f32x4*)(qb + (size_t)t * c.lds + k);
#pragma unroll
        for (int j = 0; j < 4; ++j) { sk += kv[i][j] * kv[i][j]; sq += q[j] * q[j]; }
      }
    }
    sk += __shfl_xor(sk, 1, 64); sk += __shfl_xor(sk, 2, 64);
    sq += __shfl_xor(sq, 1, 64); sq += __shfl_xor(sq, 2, 64);
    const float ik = 1.0f / sqrtf(sk + c.unit_eps);
#pragma unroll
    for (int i = 0; i < DP / 16; ++i) *(f32x4*)(ks + t * LK + 16 * i + 4 * p) = kv[i] * ik;
    if (p == 0) iq[t] = c.scale / sqrtf(sq + c.unit_eps);
  }
  __syncthreads();
  if (wave == 0) {                                    // gates of token `lane`
    const T* pr = (const T*)c.proj + (size_t)(r0 + min(lane, n - 1)) * c.ldp;
    const bool on = lane < n;
    const float beta = on ? sigmoid_f(to_f32(pr[c.o_b + h])) : 0.f;
    const T* ar = (const T*)c.ap + (size_t)(r0 + min(lane, n - 1)) * c.ldap + c.o_a;
    double g = on ? -(double)expf(c.A_log[h]) * (double)softplus_f(to_f32(ar[h]) + c.dt_bias[h]) : 0.0;
#pragma unroll
    for (int s = 1; s < 64; s *= 2) {
      const double o = __shfl_up(g, s, 64);
      if (lane >= s) g += o;
    }
    const double last = __shfl(g, 63, 64);
    const float eg = expf((float)g);
    G[lane] = g;
    be[lane] = beta;
    bg[lane] = beta * eg;
    float* f = c.fac + ((size_t)blockIdx.x * c.H + h) * DELTA_FAC;
    f[lane] = iq[lane] * eg;
    f[CH + lane] = expf((float)(last - g));
    if (lane == 0) f[2 * CH] = expf((float)last);
  }
  __syncthreads();
  if (h % (c.H / c.G) == 0) {                         // the keys transposed, once per q/k head
    float* kt = c.kt + ((size_t)blockIdx.x * c.G + gq) * DP * CH;
    for (int i = tid; i < DP * (CH / 4); i += 256) {
      const int k = i / (CH / 4), t = i % (CH / 4) * 4;
      *(f32x4*)(kt + (size_t)k * CH + t) = f32x4{ks[t * LK + k], ks[(t + 1) * LK + k], ks[(t + 2) * LK + k], ks[(t + 3) * LK + k]};
    }
  }
  // k_i . k_j (even waves) and q_i . k_j (odd waves): the ten tiles on and below the diagonal
  for (int job = wave >> 1; job < 10; job += 2) {
    const int ti = job < 1 ? 0 : (job < 3 ? 1 : (job < 6 ? 2 : 3)), tj = job - ti * (ti + 1) / 2;
    const bool isq = wave & 1;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    const float* qr = qb + (size_t)min(16 * ti + c16, n - 1) * c.lds;
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      const int k = 16 * s + 4 * g4;
      const f32x4 a = isq ? *(const f32x4*)(qr + min(k, d - 4)) : *(const f32x4*)(ks + (16 * ti + c16) * LK + k);
      acc = mfma_slice(a, *(const f32x4*)(ks + (16 * tj + c16) * LK + k), acc);
    }
    const int j = 16 * tj + c16;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * ti + 4 * g4 + r;
      const float dec = i >= j ? expf((float)(G[i] - G[j])) : 0.f;
      if (isq) {
        if (i < n) c.pm[((size_t)(r0 + i) * c.H + h) * CH + j] = iq[i] * dec * acc[r];
      } else am[i * LA + j] = i > j ? be[i] * dec * acc[r] : 0.f;
    }
  }
  __syncthreads();
  // T = (I + A)^-1: diagonal blocks by substitution, a column per lane ...
  f32x4 tb[4];                                        // block column `wave` of T; a result tile is laid out as a right operand
  {
    const int o = 16 * wave;
    float tc[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float v = i == c16 ? 1.f : 0.f;
#pragma unroll
      for (int l = 0; l < i; ++l) v = fmaf(-am[(o + i) * LA + o + l], tc[l], v);
      tc[i] = v;
    }
    f32x4 t;
#pragma unroll
    for (int r = 0; r < 4; ++r) t[r] = g4 == 0 ? tc[r] : (g4 == 1 ? tc[4 + r] : (g4 == 2 ? tc[8 + r] : tc[12 + r]));
#pragma unroll
    for (int i = 0; i < 4; ++i) tb[i] = t;            // (the places above and below the diagonal are not read before they are set)
    __syncthreads();
#pragma unroll
    for (int r = 0; r < 4; ++r) am[(o + 4 * g4 + r) * LA + o + c16] = t[r];
  }
  __syncthreads();
  // ... then block column `wave` downwards: T_ij = -T_ii sum_l A_il T_lj
#pragma unroll
  for (int i = 1; i < 4; ++i) {
    if (i <= wave) continue;
    f32x4 m = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int l = 0; l < i; ++l)
      if (l >= wave) m = mfma_slice(*(const f32x4*)(am + (16 * i + c16) * LA + 16 * l + 4 * g4), tb[l], m);
    const f32x4 z = {0.f, 0.f, 0.f, 0.f};
    tb[i] = -mfma_slice(*(const f32x4*)(am + (16 * i + c16) * LA + 16 * i + 4 * g4), m, z);
#pragma unroll
    for (int r = 0; r < 4; ++r) am[(16 * wave + 4 * g4 + r) * LA + 16 * i + c16] = tb[i][r];
  }
  __syncthreads();
  // W and U: every fourth 16-column tile per wave, all row tiles
  auto t_block = [&](int i, int l) { return *(const f32x4*)(am + (16 * l + c16) * LA + 16 * i + 4 * g4); };
  for (int ct = wave; ct < NS; ct += 4) {
    f32x4 acc[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int l = 0; l < 4; ++l) {
      f32x4 b;
#pragma unroll
      for (int j = 0; j < 4; ++j) b[j] = ks[(16 * l + 4 * g4 + j) * LK + 16 * ct + c16] * bg[16 * l + 4 * g4 + j];
#pragma unroll
      for (int i = l; i < 4; ++i) acc[i] = mfma_slice(t_block(i, l), b, acc[i]);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * i + 4 * g4 + r;
        if (t < n) c.wm[((size_t)(r0 + t) * c.H + h) * DP + 16 * ct + c16] = acc[i][r];
      }
  }
  for (int ct = wave; ct * 16 < e; ct += 4) {
    const int col = min(16 * ct + c16, e - 1);
    f32x4 acc[4], b[4];
#pragma unroll
    for (int l = 0; l < 4; ++l) {
      acc[l] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < 4; ++j) { const int t = 16 * l + 4 * g4 + j; b[l][j] = vb[(size_t)min(t, n - 1) * c.lds + col] * be[t]; }
    }
#pragma unroll
    for (int l = 0; l < 4; ++l)
#pragma unroll
      for (int i = l; i < 4; ++i) acc[i] = mfma_slice(t_block(i, l), b[l], acc[i]);
    if (16 * ct + c16 < e) {                          // (U replaces v: this wave alone reads and writes these columns)
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = 16 * i + 4 * g4 + r;
          if (t < n) vb[(size_t)t * c.lds + col] = acc[i][r];
        }
    }
  }
}

// ---- a decay per channel: grid (chunks, H), NW waves ---------------------------------------------------------------------
// T = (I + A)^-1 in place of A by the first four waves (all waves of the workgroup call this): block (i, j) of T ends up at block (j, i)
__device__ __forceinline__ void invert_chunk(float* am, int LA, int wave, int c16, int g4) {
  f32x4 tb[4];
  const int o = 16 * wave;
  if (wave < 4) {
    float tc[16], ac[16];                             // column c16 of the diagonal block, of T's and of A's
#pragma unroll
    for (int i = 0; i < 16; ++i) ac[i] = -am[(o + i) * LA + o + c16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float v = i == c16 ? 1.f : 0.f;
#pragma unroll
      for (int l = 0; l < i; ++l) v = fmaf(lane_value(ac[i], l), tc[l], v);
      tc[i] = v;
    }
    f32x4 t;
#pragma unroll
    for (int r = 0; r < 4; ++r) t[r] = g4 == 0 ? tc[r] : (g4 == 1 ? tc[4 + r] : (g4 == 2 ? tc[8 + r] : tc[12 + r]));
#pragma unroll
    for (int i = 0; i < 4; ++i) tb[i] = t;
  }
  __syncthreads();
  if (wave < 4) {
#pragma unroll
    for (int r = 0; r < 4; ++r) am[(o + 4 * g4 + r) * LA + o + c16] = tb[0][r];
  }
  __syncthreads();
  if (wave < 4) {
#pragma unroll
    for (int i = 1; i < 4; ++i) {
      if (i <= wave) continue;
      f32x4 m = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int l = 0; l < i; ++l)
        if (l >= wave) m = mfma_slice(*(const f32x4*)(am + (16 * i + c16) * LA + 16 * l + 4 * g4), tb[l], m);
      const f32x4 z = {0.f, 0.f, 0.f, 0.f};
      tb[i] = -mfma_slice(*(const f32x4*)(am + (16 * i + c16) * LA + 16 * i + 4 * g4), m, z);
#pragma unroll
      for (int r = 0; r < 4; ++r) am[(16 * wave + 4 * g4 + r) * LA + 16 * i + c16] = tb[i][r];
    }
  }
  __syncthreads();
}

// sums over the four lane groups of v[0 .. 15]: lane (c16, g4) gets those of v[4 g4 .. 4 g4 + 3].  A swap of lane halves brings both
// addends of two values' sums into place.
__device__ __forceinline__ f32x4 group_sums(const float (&v)[16]) {
  auto bits = [](float x) { return __builtin_bit_cast(uint32_t, x); };
  auto sum = [](uint32_t x, uint32_t y) { return __builtin_bit_cast(float, x) + __builtin_bit_cast(float, y); };
  // (a bit cast straight from an element of the returned vector would take the first one)
  float h[8];                                         // lanes below 32: v[r], the others: v[8 + r]
#pragma unroll
  for (int r = 0; r < 8; ++r) {
    const auto x = __builtin_amdgcn_permlane32_swap(bits(v[r]), bits(v[8 + r]), false, false);
    h[r] = sum(x[0], x[1]);
  }
  f32x4 o;                                            // odd groups take the upper half of the eight
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const auto x = __builtin_amdgcn_permlane16_swap(bits(h[r]), bits(h[4 + r]), false, false);
    o[r] = sum(x[0], x[1]);
  }
  return o;
}

// exp(-ea softplus(z)) on the hardware's exponential and logarithm: what counts is the absolute error of the exponent
__device__ __forceinline__ float decay_fast(float ea, float z) {
  constexpr float LOG2E = 1.4426950408889634f;
  const float sp2 = fmaxf(z, 0.f) * LOG2E + __builtin_amdgcn_logf(1.0f + __builtin_amdgcn_exp2f(-fabsf(z) * LOG2E));
  return __builtin_amdgcn_exp2f(-ea * sp2);
}

template <typename T, int DP, int NW>
__global__ __launch_bounds__(64 * NW) void delta_chunk_channel_kernel(DeltaCall c) {
  constexpr int NT = 64 * NW, LK = DP + 4, LA = CH + 4, NS = DP / 16, NB = NW / 4;      // NB: waves per diagonal block
  extern __shared__ __attribute__((aligned(16))) float csm[];
  float* ks = csm;                                    // [CH][LK] unit keys; from step 3 on times the decay from their block's start
  float* qs = ks + CH * LK;                           // unit queries; from step 3 on times the decay from their block's start
  float* gs = qs + CH * LK;                           // decays of the tokens; from step 3 on the unit keys times the decay to their block's end
  float* am = gs + CH * LK;                           // [CH][LA] as in delta_chunk_kernel
  float* tot = am + CH * LA;                          // [4][DP] a block's whole decay
  float* part = tot + 4 * DP;                         // [NB - 1][4][2][256] partial sums of the diagonal blocks
  __shared__ float be[CH];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c16 = lane & 15, g4 = lane >> 4;
  const int h = blockIdx.y, seg = c.t.ctile[2 * blockIdx.x], t0 = c.t.ctile[2 * blockIdx.x + 1];
  const int r0 = c.t.tok0[seg] + t0, n = min(CH, c.t.len[seg] - t0);
  const int d = c.d, e = c.e, gd = c.G * d, gq = h / (c.H / c.G);
  const float* qb = c.scan + (size_t)r0 * c.lds + gq * d;
  const float* kb = qb + gd;
  float* vb = c.scan + (size_t)r0 * c.lds + 2 * gd + (size_t)h * e;

  // 1. unit keys and queries (PT threads per token), decays; tokens beyond the end: zero vectors, decay one
  {
    constexpr int PT = NT / CH, NV = (DP + 4 * PT - 1) / (4 * PT), NG = (CH * DP / 4 + NT - 1) / NT;
    const T* ar = (const T*)c.ap + (size_t)r0 * c.ldap + c.o_a + h * d;
    float4 av[NG], bv[NG];
#pragma unroll
    for (int i = 0; i < NG; ++i) {                    // (four channels of a token; d is a multiple of four)
      const int x = min(i * NT + tid, CH * DP / 4 - 1), tt = min(x / (DP / 4), n - 1), ch = min(x % (DP / 4) * 4, d - 4);
      av[i] = load4f<T>(ar + (size_t)tt * c.ldap + ch);
      bv[i] = *(const float4*)(c.dt_bias + h * d + ch);
    }
    const int t = tid / PT, p = tid % PT;
    float sk = 0.f, sq = 0.f;
    f32x4 kv[NV], qv[NV];
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int k = 4 * (PT * i + p);
      kv[i] = qv[i] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (t < n && k < d) {
        kv[i] = *(const f32x4*)(kb + (size_t)t * c.lds + k);
        qv[i] = *(const f32x4*)(qb + (size_t)t * c.lds + k);
#pragma unroll
        for (int j = 0; j < 4; ++j) { sk += kv[i][j] * kv[i][j]; sq += qv[i][j] * qv[i][j]; }
      }
    }
#pragma unroll
    for (int s = 1; s < PT; s *= 2) { sk += __shfl_xor(sk, s, 64); sq += __shfl_xor(sq, s, 64); }
    const float ik = 1.0f / sqrtf(sk + c.unit_eps), iq = c.scale / sqrtf(sq + c.unit_eps);
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int k = 4 * (PT * i + p);
      if (k >= DP) continue;
      *(f32x4*)(ks + t * LK + k) = kv[i] * ik;
      *(f32x4*)(qs + t * LK + k) = qv[i] * iq;
    }
    const float ea = expf(c.A_log[h]);
#pragma unroll
    for (int i = 0; i < NG; ++i) {
      const int x = i * NT + tid, tt = x / (DP / 4), ch = x % (DP / 4) * 4;
      if (x >= CH * DP / 4) continue;
      const bool on = tt < n && ch < d;
      *(f32x4*)(gs + tt * LK + ch) = on ? f32x4{decay_fast(ea, av[i].x + bv[i].x), decay_fast(ea, av[i].y + bv[i].y), decay_fast(ea, av[i].z + bv[i].z),
                                                decay_fast(ea, av[i].w + bv[i].w)} : f32x4{1.f, 1.f, 1.f, 1.f};
    }
    if (tid < CH) be[tid] = tid < n ? sigmoid_f(to_f32(((const T*)c.proj)[(size_t)(r0 + tid) * c.ldp + c.o_b + h])) : 0.f;
  }
  __syncthreads();

  // 2. the blocks on the diagonal: wave w has block w mod 4 and every NB-th 16-channel slice, lane (c16, g4) column c16 and four
  // channels of a slice.  p runs down the column: k_j at token j, times a token's decay from there on (above the diagonal zero).
  const int blk = wave & 3;
  f32x4 da, dp;                                       // rows 4 g4 .. 4 g4 + 3 of column c16
  {
    float sa[16], sp[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) sa[i] = sp[i] = 0.f;
    for (int s = wave >> 2; s < NS; s += NB) {
      const int k = 16 * s + 4 * g4;
      const f32x4 kj = *(const f32x4*)(ks + (16 * blk + c16) * LK + k);
      f32x4 p = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int at = (16 * blk + i) * LK + k;
        const f32x4 g = *(const f32x4*)(gs + at), ki = *(const f32x4*)(ks + at), qi = *(const f32x4*)(qs + at);
        p *= g;
        if (i == c16) p = kj;
#pragma unroll
        for (int j = 0; j < 4; ++j) { sa[i] = fmaf(p[j], ki[j], sa[i]); sp[i] = fmaf(p[j], qi[j], sp[i]); }
        if (i % 4 == 3) asm volatile("" ::: "memory");
      }
    }
    da = group_sums(sa);
    dp = group_sums(sp);
    if (wave >= 4) {
      float* o = part + ((wave >> 2) - 1) * 2048 + blk * 512 + 4 * lane;
      *(f32x4*)o = da;
      *(f32x4*)(o + 256) = dp;
    }
  }
  __syncthreads();
  if (wave < 4) {
    for (int w = 0; w < NB - 1; ++w) {
      const float* o = part + w * 2048 + blk * 512 + 4 * lane;
      da += *(const f32x4*)o;
      dp += *(const f32x4*)(o + 256);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 4 * g4 + r, row = 16 * wave + i, col = 16 * wave + c16;
      am[row * LA + col] = i > c16 ? be[row] * da[r] : 0.f;
      if (row < n) c.pm[((size_t)(r0 + row) * c.H + h) * CH + col] = i >= c16 ? dp[r] : 0.f;
    }
  }

  // 3. decays inside the blocks: a thread per channel and block
  for (int x = tid; x < 4 * DP; x += NT) {
    const int b = x / DP, ch = x % DP, at = 16 * b * LK + ch;
    float g[16], k[16], suf = 1.f, pre = 1.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) { g[i] = gs[at + i * LK]; k[i] = ks[at + i * LK]; }
#pragma unroll
    for (int i = 15; i >= 0; --i) { gs[at + i * LK] = k[i] * suf; suf *= g[i]; }
#pragma unroll
    for (int i = 0; i < 16; ++i) { pre *= g[i]; ks[at + i * LK] = k[i] * pre; qs[at + i * LK] *= pre; }
    tot[b * DP + ch] = suf;
  }
  __syncthreads();

  // 4. the six tiles below the diagonal, of A and of P
  for (int job = wave; job < 12; job += NW) {
    const bool isq = job & 1;
    const int pr = job >> 1, ti = pr < 1 ? 1 : (pr < 3 ? 2 : 3), tj = pr - ti * (ti - 1) / 2;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    const float* left = (isq ? qs : ks) + (16 * ti + c16) * LK + 4 * g4;
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      const int k = 16 * s + 4 * g4;
      f32x4 b = *(const f32x4*)(gs + (16 * tj + c16) * LK + k);
      for (int m = tj + 1; m < ti; ++m) b *= *(const f32x4*)(tot + m * DP + k);
      acc = mfma_slice(*(const f32x4*)(left + 16 * s), b, acc);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * ti + 4 * g4 + r, j = 16 * tj + c16;
      if (isq) { if (i < n) c.pm[((size_t)(r0 + i) * c.H + h) * CH + j] = acc[r]; }
      else am[i * LA + j] = be[i] * acc[r];
    }
  }
  // what delta_carry reads besides: queries from the chunk's start, keys to the chunk's end (transposed), the chunk's decay
  for (int i = tid; i < CH * (DP / 4); i += NT) {
    const int t = i / (DP / 4), k = i % (DP / 4) * 4;
    if (t >= n) break;
    f32x4 q = *(const f32x4*)(qs + t * LK + k);
    for (int m = 0; m < t / 16; ++m) q *= *(const f32x4*)(tot + m * DP + k);
    *(f32x4*)(c.qm + ((size_t)(r0 + t) * c.H + h) * DP + k) = q;
  }
  float* kt = c.kt + ((size_t)blockIdx.x * c.H + h) * DP * CH;
  for (int i = tid; i < DP * (CH / 4); i += NT) {
    const int k = i / (CH / 4), t = i % (CH / 4) * 4;
    float f = 1.f;
    for (int m = t / 16 + 1; m < 4; ++m) f *= tot[m * DP + k];
    *(f32x4*)(kt + (size_t)k * CH + t) = f32x4{gs[t * LK + k], gs[(t + 1) * LK + k], gs[(t + 2) * LK + k], gs[(t + 3) * LK + k]} * f;
  }
  if (tid < DP) c.fac[((size_t)blockIdx.x * c.H + h) * DP + tid] = tot[tid] * tot[DP + tid] * tot[2 * DP + tid] * tot[3 * DP + tid];
  __syncthreads();

  // 5. T = (I + A)^-1, W = T diag(beta) (K with the decay from the chunk's start), U = T diag(beta) V
  invert_chunk(am, LA, wave, c16, g4);
  auto t_block = [&](int i, int l) { return *(const f32x4*)(am + (16 * l + c16) * LA + 16 * i + 4 * g4); };
  auto apply = [&](f32x4 (&acc)[4], const f32x4 (&b)[4]) {
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int l = 0; l < 4; ++l) {
#pragma unroll
      for (int i = l; i < 4; ++i) acc[i] = mfma_slice(t_block(i, l), b[l], acc[i]);
      asm volatile("" ::: "memory");
    }
  };
  auto put = [&](float* out, uint32_t ld, const f32x4 (&acc)[4]) {       // (a workgroup's outputs stay below 4 GiB)
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const uint32_t t = 16 * i + 4 * g4 + r;
        if ((int)t < n) *(float*)((char*)out + t * ld * 4u) = acc[i][r];
      }
  };
  for (int ct = wave; ct < NS; ct += NW) {
    const int col = 16 * ct + c16;
    f32x4 acc[4], b[4];
    float start = 1.f;
#pragma unroll
    for (int l = 0; l < 4; ++l) {
#pragma unroll
      for (int j = 0; j < 4; ++j) { const int t = 16 * l + 4 * g4 + j; b[l][j] = ks[t * LK + col] * start * be[t]; }
      start *= tot[l * DP + col];
    }
    apply(acc, b);
    put(c.wm + ((size_t)r0 * c.H + h) * DP + col, c.H * DP, acc);
  }
  for (int ct = (wave + NW - NS % NW) % NW; ct * 16 < e; ct += NW) {       // (beginning with the waves that had no column of W)
    const int col = min(16 * ct + c16, e - 1);
    f32x4 acc[4], b[4];
#pragma unroll
    for (int l = 0; l < 4; ++l)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int t = 16 * l + 4 * g4 + j;
        b[l][j] = *(const float*)((const char*)(vb + col) + (uint32_t)min(t, n - 1) * (uint32_t)c.lds * 4u) * be[t];
      }
    apply(acc, b);
    if (16 * ct + c16 < e) put(vb + col, c.lds, acc);  // (U replaces v: this wave alone reads and writes these columns)
  }
}

// a barrier for data in LDS alone: loads from memory stay in flight across it
__device__ __forceinline__ void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
}

// element `at` of an array that starts at a base every lane shares (32-bit byte offset: the caller keeps the arrays below 4 GiB)
template <typename V>
__device__ __forceinline__ V from_base(const float* base, uint32_t at) { return *(const V*)((const char*)base + (uint32_t)(at * 4u)); }

// grid (H, ceil(e / 16), chunk segments) -- the column groups of a head share an XCD where H is a multiple of 8 --, 8 waves on
// 16 columns of S.  Waves 0..3 carry the state (wave w: tokens 16 w .. of X, NT 16-row tiles of S), waves 4..7 make the
// outputs (tokens 16 (w - 4) ..); each SIMD has one of either, whose matrix products fill each other's waits.
// CHAN: queries and keys come with their decays, the state's decay is a number per row of S.
template <typename T, int DP, bool CHAN>
__global__ __launch_bounds__(512, 2) void delta_carry_kernel(DeltaCall c) {
  constexpr int NS = DP / 16, NT = (NS + 3) / 4, LS = DP + 4, LX = CH + 4;
  __shared__ __attribute__((aligned(16))) float st[16 * LS];     // S, [column][state row]
  __shared__ __attribute__((aligned(16))) float xt[2][16 * LX];  // X and X scaled for the state, [column][token]
  const int tid = threadIdx.x, lane = tid & 63, wave = (tid >> 6) & 3, c16 = lane & 15, g4 = lane >> 4;
  const int seg = c.t.chunk[blockIdx.z], h = blockIdx.x;
  const int row = c.t.row[seg], r0 = c.t.tok0[seg], n = c.t.len[seg], off = c.t.off[row];
  const int d = c.d, e = c.e, gd = c.G * d, gq = h / (c.H / c.G);
  const int col = blockIdx.y * 16 + c16, colc = min(col, e - 1);
  const float* scan = c.scan + (size_t)r0 * c.lds;
  constexpr int NF = CHAN ? DP : DELTA_FAC;
  const float* fb = c.fac + ((size_t)c.t.cbase[seg] * c.H + h) * NF;
  const uint32_t lds = c.lds, ldf = c.H * NF, last_chunk = (n - 1) / CH;
  auto chunk_of = [&](int t0) { return min((uint32_t)t0 / CH, last_chunk); };
  auto row_of = [&](int t0) { return (uint32_t)min(t0 + 16 * wave + c16, n - 1); };   // the token whose row of a left operand this lane feeds
  // right operand i of a step: 16 state rows / tokens of this lane's column
  auto s_slice = [&](int i) { return *(const f32x4*)(st + c16 * LS + 16 * i + 4 * g4); };

  // Every wave keeps the operands of two chunks in registers: what a half-step has used is loaded again for the chunk after the
  // next.  Loads behind the last chunk repeat its last token; where the number of chunks is odd, the last step changes nothing.
  if (tid < 256) {
    float* S = c.state + ((size_t)row * c.H + h) * (size_t)d * e;
    const bool owner = wave * NT < NS;                // (DP = 32: two waves have no tile of S)
    f32x4 s[NT];
#pragma unroll
    for (int t = 0; t < NT; ++t) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int dd = 16 * (wave * NT + t) + 4 * g4 + r;
        s[t][r] = (off > 0 && dd < d) ? S[(size_t)min(dd, d - 1) * e + colc] : 0.f;
      }
      if (owner) *(f32x4*)(st + c16 * LS + 16 * (wave * NT + t) + 4 * g4) = s[t];
    }
    struct Ops { f32x4 w[NS], kk[NT][4], fk, lr[NT]; float u[4], last; } A, B;
    const float* wb = c.wm + ((size_t)r0 * c.H + h) * DP;
    const float* ub = scan + 2 * gd + (size_t)h * e;
    const float* kb = c.kt + ((size_t)c.t.cbase[seg] * (CHAN ? c.H : c.G) + (CHAN ? h : gq)) * DP * CH;
    const uint32_t ldw = c.H * DP, ldk = (CHAN ? c.H : c.G) * DP * CH;
    auto load_first = [&](Ops& o, int t0) {
      const uint32_t at = row_of(t0) * ldw + 4 * g4, ck = chunk_of(t0) * ldf;
#pragma unroll
      for (int i = 0; i < NS; ++i) o.w[i] = from_base<f32x4>(wb, at + 16 * i);
#pragma unroll
      for (int r = 0; r < 4; ++r) o.u[r] = from_base<float>(ub, (uint32_t)min(t0 + 16 * wave + 4 * g4 + r, n - 1) * lds + colc);
      if constexpr (CHAN) {
#pragma unroll
        for (int t = 0; t < NT; ++t) o.lr[t] = from_base<f32x4>(fb, ck + min(16 * (wave * NT + t) + 4 * g4, DP - 4));
      } else {
        o.fk = from_base<f32x4>(fb, ck + CH + 16 * wave + 4 * g4);
        o.last = from_base<float>(fb, ck + 2 * CH);
      }
    };
    auto load_second = [&](Ops& o, int t0) {
      const uint32_t ck = chunk_of(t0) * ldk + 4 * g4;
#pragma unroll
      for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int i = 0; i < 4; ++i) o.kk[t][i] = from_base<f32x4>(kb, ck + min(16 * (wave * NT + t) + c16, DP - 1) * CH + 16 * i);
    };
    auto step = [&](Ops& op, int t0) {
      lds_barrier();                                  // S is complete, nobody reads X any more
      f32x4 b[NS], x[2];
#pragma unroll
      for (int i = 0; i < NS; ++i) b[i] = s_slice(i);
      x[0] = x[1] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < NS; i += 2)
#pragma unroll
        for (int j = 0; j < 4; ++j) { x[0] = mfma4(op.w[i][j], b[i][j], x[0]); x[1] = mfma4(op.w[i + 1][j], b[i + 1][j], x[1]); }
      const bool any = t0 < n;
      f32x4 xs;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        x[0][r] = op.u[r] - (x[0][r] + x[1][r]);
        if constexpr (CHAN) xs[r] = any ? x[0][r] : 0.f;
        else xs[r] = any ? x[0][r] * op.fk[r] : 0.f;  // (tokens beyond the end: their keys are zero)
      }
      *(f32x4*)(xt[0] + c16 * LX + 16 * wave + 4 * g4) = x[0];
      *(f32x4*)(xt[1] + c16 * LX + 16 * wave + 4 * g4) = xs;
      if constexpr (CHAN) {
#pragma unroll
        for (int t = 0; t < NT; ++t)
#pragma unroll
          for (int r = 0; r < 4; ++r) s[t][r] *= any ? op.lr[t][r] : 1.f;
      } else {
        const float last = any ? op.last : 1.f;
#pragma unroll
        for (int t = 0; t < NT; ++t) s[t] *= last;
      }
      load_first(op, t0 + 2 * CH);
      lds_barrier();                                  // X is complete, everybody has read S
      if (owner) {
        f32x4 xb[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) xb[i] = *(const f32x4*)(xt[1] + c16 * LX + 16 * i + 4 * g4);
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
          for (int j = 0; j < 4; ++j)
#pragma unroll
            for (int t = 0; t < NT; ++t) s[t] = mfma4(op.kk[t][i][j], xb[i][j], s[t]);
#pragma unroll
        for (int t = 0; t < NT; ++t) *(f32x4*)(st + c16 * LS + 16 * (wave * NT + t) + 4 * g4) = s[t];
      }
      load_second(op, t0 + 2 * CH);
    };
    // (in this order, so that the first waits of the loop are for the first sets alone)
    load_first(A, 0);
    asm volatile("" ::: "memory");
    load_second(A, 0);
    asm volatile("" ::: "memory");
    load_first(B, CH);
    asm volatile("" ::: "memory");
    load_second(B, CH);
    for (int t0 = 0; t0 < n; t0 += 2 * CH) {
      step(A, t0);
      step(B, t0 + CH);
    }
    if (owner && col < e) {
#pragma unroll
      for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int dd = 16 * (wave * NT + t) + 4 * g4 + r;
          if (dd < d) S[(size_t)dd * e + col] = s[t][r];
        }
    }
    put_ring<T>(c, h, gq, blockIdx.y, row, off, r0, n);
  } else {
    struct Ops { f32x4 q[NS], p[4], fq; } A, B;
    const float* qb = CHAN ? c.qm + ((size_t)r0 * c.H + h) * DP : scan + gq * d;
    const uint32_t ldq = CHAN ? c.H * DP : lds;
    const float* pb = c.pm + ((size_t)r0 * c.H + h) * CH;
    const uint32_t ldp = c.H * CH;
    auto load_first = [&](Ops& o, int t0) {
      const uint32_t at = row_of(t0) * ldq;
#pragma unroll
      for (int i = 0; i < NS; ++i) o.q[i] = from_base<f32x4>(qb, at + (CHAN ? 16 * i + 4 * g4 : min(16 * i + 4 * g4, d - 4)));   // (rows of S beyond d are zero)
      if constexpr (!CHAN) o.fq = from_base<f32x4>(fb, chunk_of(t0) * ldf + 16 * wave + 4 * g4);
    };
    auto load_second = [&](Ops& o, int t0) {
      const uint32_t at = row_of(t0) * ldp + 4 * g4;
#pragma unroll
      for (int i = 0; i < 4; ++i) o.p[i] = from_base<f32x4>(pb, at + 16 * min(i, wave));
    };
    float* ob = c.scan + (size_t)r0 * c.lds + 2 * gd + (size_t)h * e;
    auto step = [&](Ops& op, int t0) {
      lds_barrier();
      f32x4 b[NS], o[2];
#pragma unroll
      for (int i = 0; i < NS; ++i) b[i] = s_slice(i);
      o[0] = o[1] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < NS; i += 2)
#pragma unroll
        for (int j = 0; j < 4; ++j) { o[0] = mfma4(op.q[i][j], b[i][j], o[0]); o[1] = mfma4(op.q[i + 1][j], b[i + 1][j], o[1]); }
      o[0] += o[1];
      if constexpr (!CHAN) o[0] *= op.fq;
      load_first(op, t0 + 2 * CH);
      lds_barrier();
      f32x4 xb[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) xb[i] = *(const f32x4*)(xt[0] + c16 * LX + 16 * i + 4 * g4);
      o[1] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (i <= wave) o[i & 1] = mfma_slice(op.p[i], xb[i], o[i & 1]);
      o[0] += o[1];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = t0 + 16 * wave + 4 * g4 + r;
        if (t < n && col < e) ob[(uint32_t)t * lds + col] = o[0][r];
      }
      load_second(op, t0 + 2 * CH);
    };
    load_first(A, 0);
    asm volatile("" ::: "memory");
    load_second(A, 0);
    asm volatile("" ::: "memory");
    load_first(B, CH);
    asm volatile("" ::: "memory");
    load_second(B, CH);
    for (int t0 = 0; t0 < n; t0 += 2 * CH) {
      step(A, t0);
      step(B, t0 + CH);
    }
  }
}

template <typename T>
__global__ __launch_bounds__(256) void delta_out_kernel(DeltaCall c) {
  __shared__ float red[12];
  const int r = blockIdx.x;
  if (c.t.len[c.t.tok_seg[r]] < 2) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, e = c.e;
  const T* pr = (const T*)c.proj + (size_t)r * c.ldp;
  T* cat = (T*)c.cat + (size_t)r * c.ldc;
  const float* o = c.scan + (size_t)r * c.lds + 2 * c.G * c.d;
  for (int h = wave; h < c.H; h += 4) {
    float ss = 0.f;
    for (int k = lane; k < e; k += 64) { const float v = o[h * e + k]; ss += v * v; }
    const float rs = 1.0f / sqrtf(wave_sum(ss) / (float)e + c.eps);
    for (int k = lane; k < e; k += 64)
      cat[h * e + k] = from_f32<T>(o[h * e + k] * rs * c.head_norm[k] * out_gate<T>(c, r, h * e + k));
  }
  if (c.ff.ff > 0) polynorm_row<T, 256>(c.ff, pr + c.ff.in_off, cat + c.ff.out_off, red);
}

// ---- outer low-rank maps --------------------------------------------------------------------------------------------
// grid (ceil(N / 256), ceil(rows / 64)), 4 waves: a wave keeps the 64 rows of x in registers and takes every fourth 16-column tile.
// The matrix is the left operand, so a lane ends up with four neighbouring outputs of one row.
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef _Float16 f16x8 __attribute__((ext_vector_type(8)));
template <typename T>
__device__ __forceinline__ f32x4 mfma16(u32x4 a, u32x4 b, f32x4 c) {
  if constexpr (std::is_same<T, bf16>::value)
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
  else
    return __builtin_amdgcn_mfma_f32_16x16x32_f16(__builtin_bit_cast(f16x8, a), __builtin_bit_cast(f16x8, b), c, 0, 0, 0);
}
template <typename T, int KS>
__global__ __launch_bounds__(256) void low_rank_kernel(LowRankCall c) {
  constexpr int RT = 4, CT = 4;                       // row tiles, column tiles per wave
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c16 = lane & 15, g4 = lane >> 4;
  const int r0 = blockIdx.y * 64, nt = c.W.N / 16, kb = c.W.K / 32;
  int part = -1;
  u32x4 x[RT][KS];
#pragma unroll
  for (int i = 0; i < CT; ++i) {
    const int ct = blockIdx.x * 16 + i * 4 + wave;
    if (ct >= nt) break;
    const int p = ct * 16 >= c.split ? 1 : 0;
    const u32x4* w = (const u32x4*)c.W.w + ((size_t)ct * kb + p * KS) * 64 + lane;
    u32x4 a[KS];
#pragma unroll
    for (int s = 0; s < KS; ++s) a[s] = w[s * 64];
    if (p != part) {                                  // (the workgroup's first tile, and where the two halves meet)
      part = p;
#pragma unroll
      for (int t = 0; t < RT; ++t) {
        const T* src = (const T*)c.x + (size_t)min(r0 + 16 * t + c16, c.rows - 1) * c.ldx + p * c.k + 8 * g4;
#pragma unroll
        for (int s = 0; s < KS; ++s) x[t][s] = *(const u32x4*)(src + 32 * s);
      }
    }
#pragma unroll
    for (int t = 0; t < RT; ++t) {
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < KS; ++s) acc = mfma16<T>(a[s], x[t][s], acc);
      const int r = r0 + 16 * t + c16;
      const T o[4] = {from_f32<T>(acc[0]), from_f32<T>(acc[1]), from_f32<T>(acc[2]), from_f32<T>(acc[3])};
      if (r < c.rows) *(uint2*)((T*)c.out + (size_t)r * c.ldo + 16 * ct + 4 * g4) = __builtin_bit_cast(uint2, o);
    }
  }
}

template <typename T>
int low_rank_at(const LowRankCall& c, hipStream_t st) {
  const dim3 grid((c.W.N + 255) / 256, (c.rows + 63) / 64);
#define GO(KS) hipLaunchKernelGGL((low_rank_kernel<T, KS>), grid, dim3(256), 0, st, c)
  switch (c.k) { case 64: GO(2); break; case 128: GO(4); break; case 192: GO(6); break; default: GO(8); break; }
#undef GO
  MI_HIP(hipGetLastError());
  return MI_OK;
}

template <typename T>
int scanned_at(const DeltaCall& c, hipStream_t st) {
  hipLaunchKernelGGL(delta_prep_kernel<T>, dim3(c.t.R), dim3(256), 0, st, c);
  MI_HIP(hipGetLastError());
  const dim3 grid((c.e + 15) / 16, c.H, c.t.nc), block(256);
  const int dpl = (c.d + 15) / 16;
#define GO(D) do { if (c.channel) hipLaunchKernelGGL((delta_scan_kernel<T, D, true>), grid, block, 0, st, c); \
    else hipLaunchKernelGGL((delta_scan_kernel<T, D, false>), grid, block, 0, st, c); } while (0)
  if (dpl <= 1) GO(1); else if (dpl <= 2) GO(2); else if (dpl <= 4) GO(4); else if (dpl <= 6) GO(6); else if (dpl <= 8) GO(8);
  else if (dpl <= 12) GO(12); else if (dpl <= 16) GO(16); else GO(32);
#undef GO
  MI_HIP(hipGetLastError());
  return MI_OK;
}

template <typename T, int DP>
int chunked_dp(const DeltaCall& c, hipStream_t st) {
  const dim3 carry_grid(c.H, (c.e + 15) / 16, c.t.nc);
  if (c.channel) {
    constexpr int NW = DP > 64 ? 16 : 8;               // (one workgroup of 16 waves per CU, or two of 8)
    const int lds = (3 * CH * (DP + 4) + CH * (CH + 4) + 4 * DP + (NW / 4 - 1) * 2048) * (int)sizeof(float);
    MI_HIP(hipFuncSetAttribute((const void*)delta_chunk_channel_kernel<T, DP, NW>, hipFuncAttributeMaxDynamicSharedMemorySize, lds));
    hipLaunchKernelGGL((delta_chunk_channel_kernel<T, DP, NW>), dim3(c.t.nct, c.H), dim3(64 * NW), lds, st, c);
    MI_HIP(hipGetLastError());
    hipLaunchKernelGGL((delta_carry_kernel<T, DP, true>), carry_grid, dim3(512), 0, st, c);
  } else {
    const int lds = (CH * (DP + 4) + CH * (CH + 4)) * (int)sizeof(float);
    MI_HIP(hipFuncSetAttribute((const void*)delta_chunk_kernel<T, DP>, hipFuncAttributeMaxDynamicSharedMemorySize, lds));
    hipLaunchKernelGGL((delta_chunk_kernel<T, DP>), dim3(c.t.nct, c.H), dim3(256), lds, st, c);
    MI_HIP(hipGetLastError());
    hipLaunchKernelGGL((delta_carry_kernel<T, DP, false>), carry_grid, dim3(512), 0, st, c);
  }
  MI_HIP(hipGetLastError());
  return MI_OK;
}

template <typename T>
int chunked_at(const DeltaCall& c, hipStream_t st) {
  if (delta_chunk_pad(c.H, c.d, c.e, c.taps) == 0 || c.pm == nullptr || (c.channel && c.qm == nullptr) || c.lds % 4 != 0 || c.t.nct < 1)
    return fail(MI_ERR_INVALID, "delta: sizes not supported by the chunk kernels");
  const int C = 2 * c.G * c.d + c.H * c.e;
  const dim3 grid((C + 1023) / 1024, c.t.nct, CH / TW);
#define GO(K) hipLaunchKernelGGL((delta_conv_kernel<T, K>), grid, dim3(256), 0, st, c)
  switch (c.taps) { case 2: GO(2); break; case 3: GO(3); break; case 4: GO(4); break; default: GO(5); break; }
#undef GO
  MI_HIP(hipGetLastError());
  switch (delta_chunk_pad(c.H, c.d, c.e, c.taps)) {
    case 32: return chunked_dp<T, 32>(c, st);
    case 64: return chunked_dp<T, 64>(c, st);
    default: return chunked_dp<T, 128>(c, st);
  }
}

template <typename T>
int delta_at(const DeltaCall& c, hipStream_t st) {
  if (c.t.nd > 0) {
    const dim3 grid(c.t.nd, c.H + (c.ff.ff > 0 ? 1 : 0)), block(DNT);
    const int vec = c.e % 4 == 0 ? 4 : 1, slices = DNT / (c.e / vec), per = (c.d + slices - 1) / slices;
#define GO(V, M) do { if (c.channel) hipLaunchKernelGGL((delta_decode_kernel<T, V, M, true>), grid, block, 0, st, c); \
    else hipLaunchKernelGGL((delta_decode_kernel<T, V, M, false>), grid, block, 0, st, c); } while (0)
    if (vec == 4) { if (per <= 2) GO(4, 2); else if (per <= 8) GO(4, 8); else if (per <= 16) GO(4, 16); else GO(4, 0); }
    else { if (per <= 8) GO(1, 8); else GO(1, 0); }
#undef GO
    MI_HIP(hipGetLastError());
  }
  if (c.t.nc > 0) {
    if (c.wm != nullptr) MI_TRY(chunked_at<T>(c, st));
    else MI_TRY(scanned_at<T>(c, st));
    hipLaunchKernelGGL(delta_out_kernel<T>, dim3(c.t.R), dim3(256), 0, st, c);
    MI_HIP(hipGetLastError());
  }
  return MI_OK;
}

}  // namespace

int delta_chunk_pad(int H, int d, int e, int taps) {
  if (d % 4 != 0 || d > 128 || (H * e) % 4 != 0 || taps < 2 || taps > 5) return 0;
  return d <= 32 ? 32 : (d <= 64 ? 64 : 128);
}

bool delta_supported(int d, int e) { return d >= 1 && d <= 512 && e >= 1 && (e <= DNT || (e % 4 == 0 && e <= 4 * DNT)); }

bool low_rank_supported(const LowRankCall& c) {
  const bool kind = (c.W.wk == WK_BF16 && c.act == MI_BF16) || (c.W.wk == WK_F16 && c.act == MI_F16);
  return kind && c.W.layout == 1 && c.k >= 64 && c.k <= 256 && c.k % 64 == 0 && c.W.K == 2 * c.k && c.split % 16 == 0 && c.W.N % 16 == 0 &&
         c.ldx % 8 == 0 && c.ldo % 4 == 0 && c.rows > 0 && c.rows <= 65535 * 64;
}
int launch_low_rank(const LowRankCall& c, hipStream_t st) {
  if (!low_rank_supported(c)) return fail(MI_ERR_INVALID, "low_rank: shape or layout not supported");
  return c.act == MI_BF16 ? low_rank_at<bf16>(c, st) : low_rank_at<f16>(c, st);
}

int launch_delta(const DeltaCall& c, hipStream_t st) {
  if (!delta_supported(c.d, c.e) || c.taps < 1 || c.H % c.G != 0) return fail(MI_ERR_UNSUPPORTED, "delta: head sizes not supported");
  switch (c.act) {
    case MI_F32: return delta_at<float>(c, st);
    case MI_BF16: return delta_at<bf16>(c, st);
    case MI_F16: return delta_at<f16>(c, st);
  }
  return fail(MI_ERR_INVALID, "delta: bad dtype");
}

}  // namespace mi
