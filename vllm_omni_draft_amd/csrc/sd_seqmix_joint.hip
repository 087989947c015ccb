// Mechanisms of decoders whose two sublayers read the same residual through a norm each and are
// added at once (x += mixer(u + conv(u)) + ff(LN2(x)), u = LN1(x)): the residual update with both
// layer norms and the mixer's input convolution, the preparation of attention inputs that pass a
// short convolution each, a matrix memory with exponential gates (mLSTM), an activation of normed
// powers.
//
// Arithmetic as in sd_seqmix.hip: activations are f32 buffers; norms, convolutions, gates, decays
// and states are f32 always; with bf16 weights the operands of matrix products are rounded to
// bf16 where they are produced and the cache holds bf16.  Every output element is summed in an
// order fixed by the token's own position in its sequence.
//
// What a convolution needs from before a batch's rows is a state of the sequence: its last
// taps - 1 inputs, f32, oldest first ([slots, taps - 1, channels]).  `single` says that every row
// of the batch is alone in its entry (a decoding step): then the kernel that convolves a channel
// also moves its state on; otherwise a launch of its own does (conv_tail_kernel), because the
// entry's other rows still read the old state.
#include <math.h>

#include "sd_common.h"

namespace {

template <typename T> __device__ __forceinline__ float ld_f(const T* p);
template <> __device__ __forceinline__ float ld_f<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ld_f<bf16_t>(const bf16_t* p) { return (float)*p; }
template <typename T> __device__ __forceinline__ void st_f(T* p, float v);
template <> __device__ __forceinline__ void st_f<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void st_f<bf16_t>(bf16_t* p, float v) { *p = (bf16_t)v; }

__device__ __forceinline__ float sigmoid_f(float z) { return 1.f / (1.f + expf(-z)); }
__device__ __forceinline__ float log_sigmoid_f(float z) {
  return z >= 0.f ? -log1pf(expf(-z)) : z - log1pf(expf(z));
}

// Sum over a workgroup of up to 16 waves: butterfly inside each wave, then the waves in order.
__device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_sum(v);
  const int wave = threadIdx.x >> 6, n_waves = (blockDim.x + 63) >> 6;
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[wave] = v;
  __syncthreads();
  float s = red[0];
  for (int w = 1; w < n_waves; ++w) s += red[w];
  return s;
}

// N consecutive elements (N = 4: 16-byte aligned f32, 8-byte aligned bf16).
template <int N> struct Pack { float v[N]; };
template <int N, typename T> __device__ __forceinline__ Pack<N> ld_pack(const T* p);
template <> __device__ __forceinline__ Pack<1> ld_pack<1, float>(const float* p) { return {{*p}}; }
template <> __device__ __forceinline__ Pack<1> ld_pack<1, bf16_t>(const bf16_t* p) { return {{(float)*p}}; }
template <> __device__ __forceinline__ Pack<4> ld_pack<4, float>(const float* p) {
  const f32x4 v = *reinterpret_cast<const f32x4*>(p);
  return {{v[0], v[1], v[2], v[3]}};
}
template <> __device__ __forceinline__ Pack<4> ld_pack<4, bf16_t>(const bf16_t* p) {
  const bf16x4 v = *reinterpret_cast<const bf16x4*>(p);
  return {{(float)v[0], (float)v[1], (float)v[2], (float)v[3]}};
}
template <int N> __device__ __forceinline__ void st_pack(float* p, const Pack<N>& a) {
  if constexpr (N == 4) *reinterpret_cast<f32x4*>(p) = f32x4{a.v[0], a.v[1], a.v[2], a.v[3]};
  else *p = a.v[0];
}
template <int N> __device__ __forceinline__ void st_pack(bf16_t* p, const Pack<N>& a) {
  if constexpr (N == 4)
    *reinterpret_cast<bf16x4*>(p) = bf16x4{(bf16_t)a.v[0], (bf16_t)a.v[1], (bf16_t)a.v[2], (bf16_t)a.v[3]};
  else *p = (bf16_t)a.v[0];
}

// ------------------------------------------------------------------ residual update, two norms
struct JointArgs {
  float* x;                // [n, W]
  const int32_t* rows;     // or nullptr: output row i is computed from row rows[i], and x is not written
  const float* a;          // [n, W] or nullptr: added to x
  const void* a_bias;      // [W] or nullptr: added too
  float* copy;             // [n, W] or nullptr: the row afterwards
  const void* w1;          // [W] or nullptr: no norms at all
  const void* w2;          // [W] or nullptr
  float eps;
  float* h1;               // LN(x) w1, or u + conv(u) of it when conv_w; nullptr: not wanted
  bf16_t* h1_b;
  float* h2;               // LN(x) w2
  bf16_t* h2_b;
  const void* conv_w;      // [W, taps] or nullptr; rows are alone in their entries
  float* conv_state;
  const int32_t* row_pos;
  const int32_t* row_slot;
  int taps, W;
};

// A workgroup per row; a thread holds up to NV pieces of V columns in registers, so the row is read
// from memory once.
template <typename T, int V, int NV>
__global__ __launch_bounds__(1024) void joint_residual_kernel(JointArgs g) {
  __shared__ float red[16];
  const int i = blockIdx.x, W = g.W, np = W / V, nthr = blockDim.x;
  const int r = g.rows ? g.rows[i] : i;
  float* xr = g.x + (size_t)r * W;
  Pack<V> p[NV];
  float sum = 0.f;
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = (threadIdx.x + k * nthr) * V;
    if (threadIdx.x + k * nthr < np) {
      p[k] = ld_pack<V>(xr + c);
      if (g.a) {
        Pack<V> t = ld_pack<V>(g.a + (size_t)r * W + c);
        if (g.a_bias) {
          const Pack<V> b = ld_pack<V>((const T*)g.a_bias + c);
#pragma unroll
          for (int e = 0; e < V; ++e) t.v[e] += b.v[e];
        }
#pragma unroll
        for (int e = 0; e < V; ++e) p[k].v[e] += t.v[e];
        if (!g.rows) st_pack<V>(xr + c, p[k]);
      }
      if (g.copy) st_pack<V>(g.copy + (size_t)i * W + c, p[k]);
#pragma unroll
      for (int e = 0; e < V; ++e) sum += p[k].v[e];
    }
  }
  if (!g.w1) return;
  const float mean = block_sum(sum, red) / (float)W;
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < NV; ++k)
    if (threadIdx.x + k * nthr < np) {
#pragma unroll
      for (int e = 0; e < V; ++e) {
        p[k].v[e] -= mean;
        ss = fmaf(p[k].v[e], p[k].v[e], ss);
      }
    }
  const float rstd = 1.f / sqrtf(block_sum(ss, red) / (float)W + g.eps);
  const int taps = g.taps;
  const int pos = g.conv_w ? g.row_pos[r] : 0, slot = g.conv_w ? g.row_slot[r] : 0;
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    if (threadIdx.x + k * nthr >= np) continue;
    const int c = (threadIdx.x + k * nthr) * V;
    const Pack<V> w1 = ld_pack<V>((const T*)g.w1 + c);
    Pack<V> u;
#pragma unroll
    for (int e = 0; e < V; ++e) u.v[e] = p[k].v[e] * rstd * w1.v[e];
    if (g.conv_w) {
      Pack<V> acc;
#pragma unroll
      for (int e = 0; e < V; ++e) acc.v[e] = 0.f;
      const T* cw = (const T*)g.conv_w + (size_t)c * taps;
      float* st = g.conv_state + (size_t)slot * (taps - 1) * W + c;
      for (int s = 0; s < taps - 1; ++s) {     // oldest input first
        Pack<V> in = ld_pack<V>(st + (size_t)s * W);
        const bool there = pos - (taps - 1 - s) >= 0;
#pragma unroll
        for (int e = 0; e < V; ++e) {
          in.v[e] = there ? in.v[e] : 0.f;
          acc.v[e] = fmaf(ld_f(cw + e * taps + s), in.v[e], acc.v[e]);
        }
        if (s > 0) st_pack<V>(st + (size_t)(s - 1) * W, in);
      }
      if (taps > 1) st_pack<V>(st + (size_t)(taps - 2) * W, u);
#pragma unroll
      for (int e = 0; e < V; ++e) {
        acc.v[e] = fmaf(ld_f(cw + e * taps + taps - 1), u.v[e], acc.v[e]);
        u.v[e] += acc.v[e];
      }
    }
    if (g.h1) st_pack<V>(g.h1 + (size_t)i * W + c, u);
    if (g.h1_b) st_pack<V>(g.h1_b + (size_t)i * W + c, u);
    if (g.w2) {
      const Pack<V> w2 = ld_pack<V>((const T*)g.w2 + c);
      Pack<V> h;
#pragma unroll
      for (int e = 0; e < V; ++e) h.v[e] = p[k].v[e] * rstd * w2.v[e];
      if (g.h2) st_pack<V>(g.h2 + (size_t)i * W + c, h);
      if (g.h2_b) st_pack<V>(g.h2_b + (size_t)i * W + c, h);
    }
  }
}

// Rows of the entry that stand before row r in the batch, as far as the taps reach.
__device__ __forceinline__ int rows_before(const int32_t* row_slot, int r, int taps) {
  const int slot = row_slot[r];
  int t = 0;
  while (t < taps - 1 && r - t - 1 >= 0 && row_slot[r - t - 1] == slot) ++t;
  return t;
}

// out = x + conv(x): x's entry rows before r, then the sequence's state, then zeros.  A workgroup
// per (row, 256 pieces of V channels).
template <typename T, int V>
__global__ __launch_bounds__(256) void conv_add_rows_kernel(
    const float* __restrict__ x, int64_t ldx, const T* __restrict__ w, const float* __restrict__ state,
    const int32_t* __restrict__ row_pos, const int32_t* __restrict__ row_slot, float* __restrict__ out,
    bf16_t* __restrict__ out_b, int64_t ldo, int C, int taps) {
  const int r = blockIdx.x, c = (blockIdx.y * 256 + threadIdx.x) * V;
  if (c >= C) return;
  const int slot = row_slot[r], pos = row_pos[r], t = rows_before(row_slot, r, taps);
  Pack<V> acc, cur;
#pragma unroll
  for (int e = 0; e < V; ++e) acc.v[e] = cur.v[e] = 0.f;
  for (int j = taps - 1; j >= 0; --j) {
    Pack<V> in;
    if (j <= t) in = ld_pack<V>(x + (size_t)(r - j) * ldx + c);
    else if (pos - j >= 0) in = ld_pack<V>(state + ((size_t)slot * (taps - 1) + (taps - 1 - (j - t))) * C + c);
    else {
#pragma unroll
      for (int e = 0; e < V; ++e) in.v[e] = 0.f;
    }
#pragma unroll
    for (int e = 0; e < V; ++e) acc.v[e] = fmaf(ld_f(w + (size_t)(c + e) * taps + (taps - 1 - j)), in.v[e], acc.v[e]);
    if (j == 0) cur = in;
  }
#pragma unroll
  for (int e = 0; e < V; ++e) cur.v[e] += acc.v[e];
  if (out) st_pack<V>(out + (size_t)r * ldo + c, cur);
  if (out_b) st_pack<V>(out_b + (size_t)r * ldo + c, cur);
}

// An entry's last taps - 1 inputs (x + bias) become its slot's state.  A thread per channel.
template <typename T>
__global__ void conv_tail_kernel(const float* __restrict__ x, int64_t ldx, const T* __restrict__ bias,
                                 float* __restrict__ state, const int32_t* __restrict__ entries, int C, int taps) {
  const int e = blockIdx.x, c = blockIdx.y * blockDim.x + threadIdx.x;
  if (c >= C) return;
  const int slot = entries[4 * e], row0 = entries[4 * e + 1], len = entries[4 * e + 2], pos0 = entries[4 * e + 3];
  float* st = state + (size_t)slot * (taps - 1) * C + c;
  const float b = bias ? ld_f(bias + c) : 0.f;
  for (int s = 0; s < taps - 1; ++s) {   // ascending: an old input is read before its place is written
    const int at = len + s - (taps - 1);
    float v;
    if (at >= 0) v = x[(size_t)(row0 + at) * ldx + c] + b;
    else v = pos0 + at >= 0 ? st[(size_t)(len + s) * C] : 0.f;
    st[(size_t)s * C] = v;
  }
}

// ------------------------------------------------------------------ an activation of normed powers
// out = k0 N(z) + k1 N(z^2) + k2 N(z^3) + k3, z the row + bias, N(y) = y / sqrt(mean(y^2) + eps) over
// the row's F values.  By a whole workgroup.
template <typename T>
__device__ __forceinline__ void poly_norm_row(const float* __restrict__ z, const T* __restrict__ bias,
                                              const float* __restrict__ coef, float eps, int F,
                                              float* __restrict__ out, bf16_t* __restrict__ out_b, float* red) {
  constexpr int U = 8;
  const int nthr = blockDim.x;
  float s1 = 0.f, s2 = 0.f, s3 = 0.f;
  for (int c0 = threadIdx.x; c0 < F; c0 += U * nthr) {
    float v[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = c0 + u * nthr < F ? c0 + u * nthr : F - 1;
      v[u] = z[c] + (bias ? ld_f(bias + c) : 0.f);
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const float q = c0 + u * nthr < F ? v[u] * v[u] : 0.f;
      s1 += q;
      s2 = fmaf(q, q, s2);
      s3 = fmaf(q * q, q, s3);
    }
  }
  s1 = wave_sum(s1);
  s2 = wave_sum(s2);
  s3 = wave_sum(s3);
  const int wave = threadIdx.x >> 6, nw = (nthr + 63) >> 6;
  if ((threadIdx.x & 63) == 0) {
    red[wave] = s1;
    red[nw + wave] = s2;
    red[2 * nw + wave] = s3;
  }
  __syncthreads();
  s1 = red[0];
  s2 = red[nw];
  s3 = red[2 * nw];
  for (int w = 1; w < nw; ++w) {
    s1 += red[w];
    s2 += red[nw + w];
    s3 += red[2 * nw + w];
  }
  const float n = (float)F;
  const float f1 = coef[0] / sqrtf(s1 / n + eps), f2 = coef[1] / sqrtf(s2 / n + eps),
              f3 = coef[2] / sqrtf(s3 / n + eps), f0 = coef[3];
  for (int c0 = threadIdx.x; c0 < F; c0 += U * nthr) {
    float v[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = c0 + u * nthr < F ? c0 + u * nthr : F - 1;
      v[u] = z[c] + (bias ? ld_f(bias + c) : 0.f);
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = c0 + u * nthr;
      if (c < F) {
        const float o = fmaf(v[u], fmaf(v[u], fmaf(v[u], f3, f2), f1), f0);
        if (out) out[c] = o;
        if (out_b) out_b[c] = (bf16_t)o;
      }
    }
  }
}
template <typename T>
__global__ __launch_bounds__(256) void poly_norm_kernel(const float* __restrict__ z, int64_t ldz,
                                                        const T* __restrict__ bias, const float* __restrict__ coef,
                                                        float eps, int F, float* __restrict__ out,
                                                        bf16_t* __restrict__ out_b, int64_t ldo) {
  __shared__ float red[12];
  const size_t r = blockIdx.x;
  poly_norm_row<T>(z + r * ldz, bias, coef, eps, F, out ? out + r * ldo : nullptr, out_b ? out_b + r * ldo : nullptr, red);
}

// ------------------------------------------------------------------ attention inputs through convolutions
// Workgroup (r, y), a wave per unit (one head's q, k or v of a row): bias, the causal convolution
// of every channel, RMS norm with a weight per channel of the head (q and k), the query's position
// factor; q goes to q_out, k and v to the paged cache.  The last y (act.F > 0) is the row of the
// feed-forward's activation, which waits for the same product.
struct ConvPrepArgs {
  const float* proj;       // [n, ld]: channels q [H*dk], k [G*dk], v [G*dv] (k, v absent: shared)
  int64_t ld;
  const void* bias;        // [C]
  const void* conv_w;      // [C, taps]
  float* conv_state;       // [slots, taps-1, C]
  const void* q_w;         // [dk]
  const void* k_w;
  float* q_out;            // [n, H*dk]
  void* k_cache;
  void* v_cache;
  const int32_t* row_pos;
  const int32_t* row_slot;
  const int32_t* block_tables;
  float eps, temp_coef;
  int temp_every;          // 0: no position factor
  int H, G, dk, dv, shared, C, taps, single, max_blocks, page;
  int q_wgs, kv_wgs;       // workgroups per row of the q units, and of the k (or the v) units
  const float* z;          // [n, ldz] the activation's input
  int64_t ldz;
  const void* z_bias;
  const float* coef;
  float* act;              // or nullptr
  bf16_t* act_b;           // or nullptr
  int64_t ldact;
  int F;
};
constexpr int kUnitWaves = 4;
constexpr int kUnitRegs = 8;    // channels per lane at most: a head has up to 512

template <typename T>
__global__ __launch_bounds__(256) void conv_prep_kernel(ConvPrepArgs g) {
  __shared__ float red[12];
  const int r = blockIdx.x, y = blockIdx.y;
  const int n_wgs = g.q_wgs + (g.shared ? 0 : 2 * g.kv_wgs);
  if (y >= n_wgs) {
    poly_norm_row<T>(g.z + (size_t)r * g.ldz, (const T*)g.z_bias, g.coef, g.eps, g.F,
                     g.act ? g.act + (size_t)r * g.ldact : nullptr, g.act_b ? g.act_b + (size_t)r * g.ldact : nullptr, red);
    return;
  }
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int kind = y < g.q_wgs ? 0 : (y < g.q_wgs + g.kv_wgs ? 1 : 2);   // q, k, v
  const int unit = (kind == 0 ? y : (kind == 1 ? y - g.q_wgs : y - g.q_wgs - g.kv_wgs)) * kUnitWaves + wave;
  if (unit >= (kind == 0 ? g.H : g.G)) return;
  const int d = kind == 2 ? g.dv : g.dk;
  const int ch0 = (kind == 0 ? 0 : (kind == 1 ? g.H * g.dk : (g.H + g.G) * g.dk)) + unit * d;
  const int pos = g.row_pos[r], slot = g.row_slot[r], taps = g.taps;
  const int t = g.single ? 0 : rows_before(g.row_slot, r, taps);
  const float* pr = g.proj + (size_t)r * g.ld + ch0;
  const T* bias = (const T*)g.bias;
  const T* cw = (const T*)g.conv_w;
  float* st = g.conv_state + (size_t)slot * (taps - 1) * g.C + ch0;
  float val[kUnitRegs];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < kUnitRegs; ++k) {
    const int c = lane + 64 * k;
    val[k] = 0.f;
    if (c < d) {
      const float b = bias ? ld_f(bias + ch0 + c) : 0.f;
      float acc = 0.f, in = 0.f;
      for (int j = taps - 1; j >= 0; --j) {
        if (j <= t) in = pr[c - (int64_t)j * g.ld] + b;
        else if (pos - j >= 0) in = st[(size_t)(taps - 1 - (j - t)) * g.C + c];
        else in = 0.f;
        acc = fmaf(ld_f(cw + (size_t)(ch0 + c) * taps + (taps - 1 - j)), in, acc);
        // (a row alone in its entry: inputs move one place towards the oldest as they are read)
        if (g.single && j < taps - 1) st[(size_t)(taps - 2 - j) * g.C + c] = in;
      }
      val[k] = acc;
      ss = fmaf(acc, acc, ss);
    }
  }
  if (kind < 2) {
    float f = 1.f / sqrtf(wave_sum(ss) / (float)d + g.eps);
    const T* w = (const T*)(kind == 0 ? g.q_w : g.k_w);
    const float temp = kind == 0 && g.temp_every > 0
                           ? 1.f + g.temp_coef * logf((float)((pos + 1) / g.temp_every) + 1.f) : 1.f;
#pragma unroll
    for (int k = 0; k < kUnitRegs; ++k) {
      const int c = lane + 64 * k;
      if (c < d) val[k] = val[k] * f * ld_f(w + c) * temp;
    }
  }
  if (kind == 0) {
    float* q = g.q_out + (size_t)r * g.H * g.dk + unit * d;
#pragma unroll
    for (int k = 0; k < kUnitRegs; ++k)
      if (lane + 64 * k < d) q[lane + 64 * k] = val[k];
    return;
  }
  const int pg = g.block_tables[(size_t)slot * g.max_blocks + pos / g.page];
  T* dst = (T*)(kind == 1 ? g.k_cache : g.v_cache) + (((size_t)pg * g.G + unit) * g.page + pos % g.page) * d;
#pragma unroll
  for (int k = 0; k < kUnitRegs; ++k)
    if (lane + 64 * k < d) st_f(dst + lane + 64 * k, val[k]);
}

// ------------------------------------------------------------------ matrix memory with exponential gates
// Per head, token by token, with log gates i = cap tanh((z_i + b_i) / cap), f = logsigmoid(cap
// tanh((z_f + b_f) / cap)) and a running maximum m (0 at the start):
//   m' = max(f + m, i);  S <- e^(f + m - m') S + e^(i - m') k v^T;  n <- the same with k alone
// num[t] = S^T q (dv columns) and, in column dv, n . q; m_rows[t] = m'.  Columns are tiled over
// workgroups (the normalizer is one more column, whose value is 1); every workgroup forms the gates
// itself.  A thread owns 16 consecutive key channels of one column; strips' partial dot products
// are added in strip order.  m's state is left to the launch that reads m_rows (a workgroup of
// another tile may still have to read the old one).
constexpr int kStrip = 16;
constexpr int kScanLoads = 8;
constexpr int kScanLoadsV = 16;
constexpr int kScanChunk = 16;
struct MlstmArgs {
  const float* q;          // [n, ld] H*dk channels each
  const float* k;
  const float* v;          // [n, ld] H*dv channels
  const float* zi;         // [n, ld] H
  const float* zf;
  int64_t ld;
  const float* bi;         // [H]
  const float* bf;
  float cap, q_scale;
  float* S;                // [slots, H, dk, dv]
  float* nrm;              // [slots, H, dk]
  float* m;                // [slots, H]
  const int32_t* entries;
  float* num;              // [n, H, dv + 1]
  float* m_rows;           // [n, H]
  int H, dk, dv;
};
__global__ __launch_bounds__(256) void mlstm_scan_kernel(MlstmArgs g, int CT, int NS, int CH) {
  extern __shared__ float lds[];
  const int dk = g.dk, dv = g.dv, H = g.H, dkp = NS * kStrip;
  float* qs = lds;                  // [CH][dkp]
  float* ks = qs + CH * dkp;        // [CH][dkp]
  float* vs = ks + CH * dkp;        // [CH][CT]
  float* dsc = vs + CH * CT;        // [CH] decay
  float* asc = dsc + CH;            // [CH] key factor
  float* part = asc + CH;           // [CH][NS][CT]
  const int tid = threadIdx.x, nthr = CT * NS;
  const int c = tid % CT, s = tid / CT;
  const int h = blockIdx.y, e = blockIdx.z;
  const int col = blockIdx.x * CT + c;
  const int slot = g.entries[4 * e], row0 = g.entries[4 * e + 1], len = g.entries[4 * e + 2], pos0 = g.entries[4 * e + 3];
  float* st = col < dv ? g.S + (((size_t)slot * H + h) * dk) * dv + col : g.nrm + ((size_t)slot * H + h) * dk;
  const int st_row = col < dv ? dv : 1;
  const bool live = col <= dv;
  const int r0 = s * kStrip;
  float S[kStrip];
#pragma unroll
  for (int r = 0; r < kStrip; ++r)
    S[r] = (pos0 > 0 && r0 + r < dk && live) ? st[(size_t)(r0 + r) * st_row] : 0.f;
  float m_run = pos0 > 0 ? g.m[(size_t)slot * H + h] : 0.f;
  const float bi = g.bi[h], bf = g.bf[h], cap = g.cap;
  float pq[kScanLoads], pk[kScanLoads], pv[kScanLoadsV], pi = 0.f, pf = 0.f;
  auto fetch = [&](int t0) {
    const int nt = len - t0 < CH ? len - t0 : CH;
#pragma unroll
    for (int i = 0; i < kScanLoads; ++i) {
      const int idx = tid + i * nthr;
      const int t = idx / dkp, ch = idx % dkp;
      const bool in = idx < nt * dkp && ch < dk;
      // (every load is issued, on an address clamped into the chunk)
      const int tc = t < nt ? t : nt - 1, cc = ch < dk ? ch : dk - 1;
      const size_t at = (size_t)(row0 + t0 + tc) * g.ld + (size_t)h * dk + cc;
      const float lq = g.q[at], lk = g.k[at];
      pq[i] = in ? lq * g.q_scale : 0.f;
      pk[i] = in ? lk : 0.f;
    }
#pragma unroll
    for (int i = 0; i < kScanLoadsV; ++i) {
      const int idx = tid + i * nthr;
      const int t = idx / CT, vcol = blockIdx.x * CT + idx % CT;
      const bool in = idx < nt * CT;
      const int tc = t < nt ? t : nt - 1, vc = vcol < dv ? vcol : dv - 1;
      const float lv = g.v[(size_t)(row0 + t0 + tc) * g.ld + (size_t)h * dv + vc];
      pv[i] = !in ? 0.f : (vcol < dv ? lv : (vcol == dv ? 1.f : 0.f));
    }
    const int tc = tid < nt ? tid : nt - 1;
    pi = g.zi[(size_t)(row0 + t0 + tc) * g.ld + h] + bi;
    pf = g.zf[(size_t)(row0 + t0 + tc) * g.ld + h] + bf;
  };
  fetch(0);
  for (int t0 = 0; t0 < len; t0 += CH) {
    const int nt = len - t0 < CH ? len - t0 : CH;
#pragma unroll
    for (int i = 0; i < kScanLoads; ++i) {
      const int idx = tid + i * nthr;
      if (idx < CH * dkp) {
        qs[idx] = pq[i];
        ks[idx] = pk[i];
      }
    }
#pragma unroll
    for (int i = 0; i < kScanLoadsV; ++i) {
      const int idx = tid + i * nthr;
      if (idx < CH * CT) vs[idx] = pv[i];
    }
    if (tid < SD_WAVE) {   // the first wave forms the chunk's gates, a lane per token
      const float li = cap * tanhf(pi / cap), lf = log_sigmoid_f(cap * tanhf(pf / cap));
      float m = m_run, d = 0.f, a = 0.f, mine = 0.f;
      for (int t = 0; t < nt; ++t) {
        const float f_t = __shfl(lf, t, SD_WAVE), i_t = __shfl(li, t, SD_WAVE);
        const float m_new = fmaxf(f_t + m, i_t);
        if (t == tid) {
          d = expf(f_t + m - m_new);
          a = expf(i_t - m_new);
          mine = m_new;
        }
        m = m_new;
      }
      m_run = m;
      if (tid < nt) {
        dsc[tid] = d;
        asc[tid] = a;
        if (blockIdx.x == 0) g.m_rows[(size_t)(row0 + t0 + tid) * H + h] = mine;
      }
    }
    __syncthreads();
    if (t0 + CH < len) fetch(t0 + CH);
    for (int t = 0; t < nt; ++t) {
      const float d = dsc[t], av = asc[t] * vs[t * CT + c];
      const float* qt = qs + t * dkp + r0;
      const float* kt = ks + t * dkp + r0;
      float acc = 0.f;
#pragma unroll
      for (int r = 0; r < kStrip; ++r) {
        S[r] = fmaf(d, S[r], kt[r] * av);
        acc = fmaf(S[r], qt[r], acc);
      }
      part[(t * NS + s) * CT + c] = acc;
    }
    __syncthreads();
    for (int idx = tid; idx < nt * CT; idx += nthr) {
      const int t = idx / CT, cc = idx % CT;
      const int ocol = blockIdx.x * CT + cc;
      if (ocol > dv) continue;
      float o = part[(t * NS) * CT + cc];
      for (int ss = 1; ss < NS; ++ss) o += part[(t * NS + ss) * CT + cc];
      g.num[((size_t)(row0 + t0 + t) * H + h) * (dv + 1) + ocol] = o;
    }
  }
  if (live) {
#pragma unroll
    for (int r = 0; r < kStrip; ++r)
      if (r0 + r < dk) st[(size_t)(r0 + r) * st_row] = S[r];
  }
}

// Read-out, a wave per (row, head): o = num / (max(|n . q|, e^-m) + 1e-6), divided by its root mean
// square over the head, times w (a weight per channel of all heads), times sigmoid(gate).  The
// last row of an entry leaves its m in the slot's state.  The last y is the feed-forward's
// activation, as in conv_prep_kernel.
struct MlstmPostArgs {
  const float* num;
  const float* m_rows;
  float* m;                // [slots, H]
  const int32_t* row_slot;
  const float* gate;       // [n, ldg] H*dv
  int64_t ldg;
  const void* w;           // [H*dv]
  float eps;
  float* y;                // or nullptr
  bf16_t* y_b;             // or nullptr
  int64_t ldy;
  int H, dv, wgs;
  const float* z;
  int64_t ldz;
  const void* z_bias;
  const float* coef;
  float* act;
  bf16_t* act_b;
  int F;
};
template <typename T>
__global__ __launch_bounds__(256) void mlstm_post_kernel(MlstmPostArgs g) {
  __shared__ float red[12];
  const int r = blockIdx.x;
  if ((int)blockIdx.y >= g.wgs) {
    poly_norm_row<T>(g.z + (size_t)r * g.ldz, (const T*)g.z_bias, g.coef, g.eps, g.F,
                     g.act ? g.act + (size_t)r * g.ldy : nullptr, g.act_b ? g.act_b + (size_t)r * g.ldy : nullptr, red);
    return;
  }
  const int h = blockIdx.y * kUnitWaves + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (h >= g.H) return;
  const int dv = g.dv;
  const float* num = g.num + ((size_t)r * g.H + h) * (dv + 1);
  const float m = g.m_rows[(size_t)r * g.H + h];
  const float inv = 1.f / (fmaxf(fabsf(num[dv]), expf(-m)) + 1e-6f);
  float val[kUnitRegs];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < kUnitRegs; ++k) {
    const int c = lane + 64 * k;
    val[k] = c < dv ? num[c] * inv : 0.f;
    ss = fmaf(val[k], val[k], ss);
  }
  const float rstd = 1.f / sqrtf(wave_sum(ss) / (float)dv + g.eps);
#pragma unroll
  for (int k = 0; k < kUnitRegs; ++k) {
    const int c = lane + 64 * k;
    if (c < dv) {
      const int ch = h * dv + c;
      const float o = val[k] * rstd * ld_f((const T*)g.w + ch) * sigmoid_f(g.gate[(size_t)r * g.ldg + ch]);
      if (g.y) g.y[(size_t)r * g.ldy + ch] = o;
      if (g.y_b) g.y_b[(size_t)r * g.ldy + ch] = (bf16_t)o;
    }
  }
  const int slot = g.row_slot[r];
  if (lane == 0 && (r + 1 == (int)gridDim.x || g.row_slot[r + 1] != slot)) g.m[(size_t)slot * g.H + h] = m;
}

template <typename T>
void launch_joint(const JointArgs& g, int n, hipStream_t st) {
  const bool quad = g.W % 4 == 0;
  const int np = quad ? g.W / 4 : g.W;
  int nthr = (np + 63) / 64 * 64;
  if (nthr > 1024) nthr = 1024;
  if (quad) {
    if (np <= nthr) joint_residual_kernel<T, 4, 1><<<n, nthr, 0, st>>>(g);
    else joint_residual_kernel<T, 4, 4><<<n, nthr, 0, st>>>(g);
  } else {
    if (np <= 4 * nthr) joint_residual_kernel<T, 1, 4><<<n, nthr, 0, st>>>(g);
    else joint_residual_kernel<T, 1, 16><<<n, nthr, 0, st>>>(g);
  }
}

}  // namespace

// ====================================================================== C entry points
extern "C" int sd_joint_residual(float* x, const int32_t* rows, const float* a, const void* a_bias, float* x_copy,
                                 const void* w1, const void* w2, int w_f32, float eps, float* h1, void* h1_bf16,
                                 float* h2, void* h2_bf16, const void* conv_w, int taps, float* conv_state,
                                 const int32_t* row_pos, const int32_t* row_slot, int n_rows, int W,
                                 sd_stream_t stream) {
  SD_REQUIRE(x && n_rows >= 1 && W >= 1 && (!a_bias || a) && (!w2 || w1), SD_ERR_INVALID, "sd_joint_residual: bad argument");
  SD_REQUIRE(W <= 16384, SD_ERR_UNSUPPORTED, "sd_joint_residual: width %d above 16384", W);
  SD_REQUIRE(!conv_w || (w1 && taps >= 1 && (taps == 1 || conv_state) && row_pos && row_slot && !rows), SD_ERR_INVALID,
             "sd_joint_residual: a convolution needs its state, positions and slots, and no row list");
  JointArgs g{x, rows, a, a_bias, x_copy, w1, w2, eps, h1, (bf16_t*)h1_bf16, h2, (bf16_t*)h2_bf16, conv_w, conv_state,
              row_pos, row_slot, taps, W};
  if (w_f32) launch_joint<float>(g, n_rows, (hipStream_t)stream);
  else launch_joint<bf16_t>(g, n_rows, (hipStream_t)stream);
  SD_CHECK_LAUNCH("sd_joint_residual");
  return SD_OK;
}

extern "C" int sd_conv_tail(const float* x, int64_t ldx, const void* bias, int w_f32, float* conv_state,
                            const int32_t* entries, int n_entries, int C, int taps, sd_stream_t stream) {
  SD_REQUIRE(x && entries && n_entries >= 1 && C >= 1 && taps >= 1 && (taps == 1 || conv_state) && ldx >= C,
             SD_ERR_INVALID, "sd_conv_tail: bad argument");
  if (taps == 1) return SD_OK;
  dim3 grid(n_entries, (C + 255) / 256);
  hipStream_t st = (hipStream_t)stream;
  if (w_f32) conv_tail_kernel<float><<<grid, 256, 0, st>>>(x, ldx, (const float*)bias, conv_state, entries, C, taps);
  else conv_tail_kernel<bf16_t><<<grid, 256, 0, st>>>(x, ldx, (const bf16_t*)bias, conv_state, entries, C, taps);
  SD_CHECK_LAUNCH("sd_conv_tail");
  return SD_OK;
}

extern "C" int sd_conv_add_rows(const float* x, int64_t ldx, const void* w, int w_f32, float* conv_state,
                                const int32_t* row_pos, const int32_t* row_slot, const int32_t* entries,
                                int n_entries, float* out, void* out_bf16, int64_t ldo, int n_rows, int C, int taps,
                                sd_stream_t stream) {
  SD_REQUIRE(x && w && row_pos && row_slot && entries && (out || out_bf16) && n_entries >= 1 && n_rows >= 1 && C >= 1 &&
                 taps >= 1 && (taps == 1 || conv_state) && ldx >= C && ldo >= C && out != x,
             SD_ERR_INVALID, "sd_conv_add_rows: bad argument");
  hipStream_t st = (hipStream_t)stream;
  const bool quad = C % 4 == 0 && ldx % 4 == 0 && ldo % 4 == 0;
  dim3 grid(n_rows, ((quad ? C / 4 : C) + 255) / 256);
#define SD_GO(T, V) conv_add_rows_kernel<T, V><<<grid, 256, 0, st>>>(x, ldx, (const T*)w, conv_state, row_pos, row_slot, out, (bf16_t*)out_bf16, ldo, C, taps)
  if (w_f32) { if (quad) SD_GO(float, 4); else SD_GO(float, 1); }
  else { if (quad) SD_GO(bf16_t, 4); else SD_GO(bf16_t, 1); }
#undef SD_GO
  SD_CHECK_LAUNCH("sd_conv_add_rows");
  return sd_conv_tail(x, ldx, nullptr, w_f32, conv_state, entries, n_entries, C, taps, stream);
}

extern "C" int sd_poly_norm_rows(const float* z, int64_t ldz, const void* bias, int w_f32, const float* coef, float eps,
                                 float* out, void* out_bf16, int64_t ldo, int n_rows, int F, sd_stream_t stream) {
  SD_REQUIRE(z && coef && (out || out_bf16) && n_rows >= 1 && F >= 1 && ldz >= F && ldo >= F, SD_ERR_INVALID,
             "sd_poly_norm_rows: bad argument");
  hipStream_t st = (hipStream_t)stream;
  if (w_f32) poly_norm_kernel<float><<<n_rows, 256, 0, st>>>(z, ldz, (const float*)bias, coef, eps, F, out, (bf16_t*)out_bf16, ldo);
  else poly_norm_kernel<bf16_t><<<n_rows, 256, 0, st>>>(z, ldz, (const bf16_t*)bias, coef, eps, F, out, (bf16_t*)out_bf16, ldo);
  SD_CHECK_LAUNCH("sd_poly_norm_rows");
  return SD_OK;
}

extern "C" int sd_conv_attn_prep(const float* proj, int64_t ld, const void* bias, const void* conv_w, int taps,
                                 float* conv_state, int H, int G, int dk, int dv, int shared, const void* q_norm_w,
                                 const void* k_norm_w, int w_f32, float eps, float temp_coef, int temp_every,
                                 float* q_out, void* k_cache, void* v_cache, const int32_t* row_pos,
                                 const int32_t* row_slot, const int32_t* entries, int n_entries,
                                 const int32_t* block_tables, int max_blocks, int page, int n_rows,
                                 const sd_poly_norm* act, sd_stream_t stream) {
  SD_REQUIRE(proj && conv_w && q_norm_w && q_out && row_pos && row_slot && entries && n_entries >= 1 &&
                 n_rows >= n_entries && H >= 1 && G >= 1 && H % G == 0 && dk >= 1 && dv >= 1 && taps >= 1 &&
                 (taps == 1 || conv_state) && temp_every >= 0,
             SD_ERR_INVALID, "sd_conv_attn_prep: bad argument");
  SD_REQUIRE(dk <= 64 * kUnitRegs && dv <= 64 * kUnitRegs, SD_ERR_UNSUPPORTED, "sd_conv_attn_prep: dim %d / vdim %d above 512", dk, dv);
  SD_REQUIRE(shared || (k_norm_w && k_cache && v_cache && block_tables && max_blocks >= 1 && page >= 1), SD_ERR_INVALID,
             "sd_conv_attn_prep: keys and values need their norm, caches and block tables");
  ConvPrepArgs g{};
  g.proj = proj; g.ld = ld; g.bias = bias; g.conv_w = conv_w; g.conv_state = conv_state; g.q_w = q_norm_w; g.k_w = k_norm_w;
  g.q_out = q_out; g.k_cache = k_cache; g.v_cache = v_cache; g.row_pos = row_pos; g.row_slot = row_slot;
  g.block_tables = block_tables; g.eps = eps; g.temp_coef = temp_coef; g.temp_every = temp_every;
  g.H = H; g.G = G; g.dk = dk; g.dv = dv; g.shared = shared; g.taps = taps; g.single = n_rows == n_entries;
  g.C = H * dk + (shared ? 0 : G * (dk + dv));
  g.max_blocks = max_blocks; g.page = page;
  SD_REQUIRE(ld >= g.C, SD_ERR_INVALID, "sd_conv_attn_prep: ld < channels");
  g.q_wgs = (H + kUnitWaves - 1) / kUnitWaves;
  g.kv_wgs = (G + kUnitWaves - 1) / kUnitWaves;
  if (act) {
    SD_REQUIRE(act->z && act->coef && (act->out || act->out_bf16) && act->n >= 1 && act->ldz >= act->n && act->ldo >= act->n,
               SD_ERR_INVALID, "sd_conv_attn_prep: bad activation");
    g.z = act->z; g.ldz = act->ldz; g.z_bias = act->bias; g.coef = act->coef; g.act = act->out;
    g.act_b = (bf16_t*)act->out_bf16; g.ldact = act->ldo; g.F = act->n;
  }
  dim3 grid(n_rows, g.q_wgs + (shared ? 0 : 2 * g.kv_wgs) + (act ? 1 : 0));
  hipStream_t st = (hipStream_t)stream;
  if (w_f32) conv_prep_kernel<float><<<grid, 256, 0, st>>>(g);
  else conv_prep_kernel<bf16_t><<<grid, 256, 0, st>>>(g);
  SD_CHECK_LAUNCH("sd_conv_attn_prep");
  if (g.single) return SD_OK;
  return sd_conv_tail(proj, ld, bias, w_f32, conv_state, entries, n_entries, g.C, taps, stream);
}

extern "C" int sd_mlstm_scan(const float* q, const float* k, const float* v, const float* zi, const float* zf,
                             int64_t ld, const float* bi, const float* bf, float cap, float q_scale, float* S,
                             float* n_state, const float* m_state, const int32_t* entries, int n_entries, float* num,
                             float* m_rows, int H, int dk, int dv, sd_stream_t stream) {
  SD_REQUIRE(q && k && v && zi && zf && bi && bf && S && n_state && m_state && entries && num && m_rows &&
                 n_entries >= 1 && H >= 1 && dv >= 1 && cap > 0.f,
             SD_ERR_INVALID, "sd_mlstm_scan: bad argument");
  SD_REQUIRE(dk >= 1 && dk <= 256, SD_ERR_UNSUPPORTED, "sd_mlstm_scan: key size %d outside 1..256", dk);
  const int NS = (dk + kStrip - 1) / kStrip, cols = dv + 1;
  int CT = 256 / NS;
  if (CT > cols) CT = cols;
  if (CT > 64) CT = 64;
  const int dkp = NS * kStrip;
  int CH = kScanLoads * (CT * NS) / dkp;   // a chunk's q / k elements fit kScanLoads per thread
  if (CH > kScanChunk) CH = kScanChunk;
  if (CH > CT * NS) CH = CT * NS;          // a lane per token of the chunk forms the gates
  SD_REQUIRE(CH >= 1 && CH * CT <= kScanLoadsV * CT * NS, SD_ERR_UNSUPPORTED,
             "sd_mlstm_scan: key size %d with value size %d leaves no chunk", dk, dv);
  const size_t lds = sizeof(float) * ((size_t)2 * CH * dkp + (size_t)CH * CT + 2 * CH + (size_t)CH * NS * CT);
  MlstmArgs g{q, k, v, zi, zf, ld, bi, bf, cap, q_scale, S, n_state, const_cast<float*>(m_state), entries, num, m_rows, H, dk, dv};
  mlstm_scan_kernel<<<dim3((cols + CT - 1) / CT, H, n_entries), CT * NS, lds, (hipStream_t)stream>>>(g, CT, NS, CH);
  SD_CHECK_LAUNCH("sd_mlstm_scan");
  return SD_OK;
}

extern "C" int sd_mlstm_read(const float* num, const float* m_rows, float* m_state, const int32_t* row_slot,
                             const float* gate, int64_t ldg, const void* w, int w_f32, float eps, float* y,
                             void* y_bf16, int64_t ldy, int n_rows, int H, int dv, const sd_poly_norm* act,
                             sd_stream_t stream) {
  SD_REQUIRE(num && m_rows && m_state && row_slot && gate && w && (y || y_bf16) && n_rows >= 1 && H >= 1 && dv >= 1 &&
                 ldg >= (int64_t)H * dv && ldy >= (int64_t)H * dv,
             SD_ERR_INVALID, "sd_mlstm_read: bad argument");
  SD_REQUIRE(dv <= 64 * kUnitRegs, SD_ERR_UNSUPPORTED, "sd_mlstm_read: value size %d above 512", dv);
  MlstmPostArgs g{};
  g.num = num; g.m_rows = m_rows; g.m = m_state; g.row_slot = row_slot; g.gate = gate; g.ldg = ldg; g.w = w; g.eps = eps;
  g.y = y; g.y_b = (bf16_t*)y_bf16; g.ldy = ldy; g.H = H; g.dv = dv; g.wgs = (H + kUnitWaves - 1) / kUnitWaves;
  if (act) {
    SD_REQUIRE(act->z && act->coef && (act->out || act->out_bf16) && act->n >= 1 && act->ldz >= act->n && act->ldo == ldy,
               SD_ERR_INVALID, "sd_mlstm_read: bad activation");
    g.z = act->z; g.ldz = act->ldz; g.z_bias = act->bias; g.coef = act->coef; g.act = act->out;
    g.act_b = (bf16_t*)act->out_bf16; g.F = act->n;
  }
  dim3 grid(n_rows, g.wgs + (act ? 1 : 0));
  hipStream_t st = (hipStream_t)stream;
  if (w_f32) mlstm_post_kernel<float><<<grid, 256, 0, st>>>(g);
  else mlstm_post_kernel<bf16_t><<<grid, 256, 0, st>>>(g);
  SD_CHECK_LAUNCH("sd_mlstm_read");
  return SD_OK;
}
