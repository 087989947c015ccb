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

#include <mutex>

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
  const void* conv_w;      // [taps, W] or nullptr; rows are alone in their entries
  float* conv_state;
  const int32_t* row_pos;
  const int32_t* row_slot;
  int taps, W;
};

// A workgroup per row; a thread holds up to NV pieces of V columns in registers, so the row is read
// from memory once.  With one piece per thread and few taps everything the end of the kernel needs
// (norm weights, convolution, state) is asked for before the row's sums are formed.
constexpr int kEarlyTaps = 4;
template <typename T, int V, int NV>
__global__ __launch_bounds__(1024) void joint_residual_kernel(JointArgs g) {
  __shared__ float red[16];
  const int i = blockIdx.x, W = g.W, np = W / V, nthr = blockDim.x, taps = g.taps;
  const int r = g.rows ? g.rows[i] : i;
  const int pos = g.conv_w ? g.row_pos[r] : 0, slot = g.conv_w ? g.row_slot[r] : 0;
  float* xr = g.x + (size_t)r * W;
  const bool early = NV == 1 && taps <= kEarlyTaps;
  Pack<V> w1e, w2e, cwe[kEarlyTaps], ste[kEarlyTaps - 1];
  if (early && g.w1 && (int)threadIdx.x < np) {
    const int c = threadIdx.x * V;
    w1e = ld_pack<V>((const T*)g.w1 + c);
    if (g.w2) w2e = ld_pack<V>((const T*)g.w2 + c);
    if (g.conv_w) {
#pragma unroll
      for (int t = 0; t < kEarlyTaps; ++t)
        if (t < taps) cwe[t] = ld_pack<V>((const T*)g.conv_w + (size_t)t * W + c);
#pragma unroll
      for (int t = 0; t < kEarlyTaps - 1; ++t)
        if (t < taps - 1) ste[t] = ld_pack<V>(g.conv_state + ((size_t)slot * (taps - 1) + t) * W + c);
    }
  }
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
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    if (threadIdx.x + k * nthr >= np) continue;
    const int c = (threadIdx.x + k * nthr) * V;
    const Pack<V> w1 = early ? w1e : ld_pack<V>((const T*)g.w1 + c);
    Pack<V> u;
#pragma unroll
    for (int e = 0; e < V; ++e) u.v[e] = p[k].v[e] * rstd * w1.v[e];
    if (g.conv_w) {   // oldest input first; inputs move one place towards the oldest
      Pack<V> acc;
#pragma unroll
      for (int e = 0; e < V; ++e) acc.v[e] = 0.f;
      float* st = g.conv_state + (size_t)slot * (taps - 1) * W + c;
      auto tap = [&](int t, Pack<V> in, const Pack<V>& cw) {
        const bool there = pos - (taps - 1 - t) >= 0;
#pragma unroll
        for (int e = 0; e < V; ++e) {
          in.v[e] = there ? in.v[e] : 0.f;
          acc.v[e] = fmaf(cw.v[e], in.v[e], acc.v[e]);
        }
        if (t > 0) st_pack<V>(st + (size_t)(t - 1) * W, in);
      };
      Pack<V> cw;
      if (early) {
#pragma unroll
        for (int t = 0; t < kEarlyTaps - 1; ++t)
          if (t < taps - 1) tap(t, ste[t], cwe[t]);
        cw = cwe[0];
#pragma unroll
        for (int t = 1; t < kEarlyTaps; ++t)
          if (t == taps - 1) cw = cwe[t];
      } else {
        for (int t = 0; t < taps - 1; ++t)
          tap(t, ld_pack<V>(st + (size_t)t * W), ld_pack<V>((const T*)g.conv_w + (size_t)t * W + c));
        cw = ld_pack<V>((const T*)g.conv_w + (size_t)(taps - 1) * W + c);
      }
      if (taps > 1) st_pack<V>(st + (size_t)(taps - 2) * W, u);
#pragma unroll
      for (int e = 0; e < V; ++e) {
        acc.v[e] = fmaf(cw.v[e], u.v[e], acc.v[e]);
        u.v[e] += acc.v[e];
      }
    }
    if (g.h1) st_pack<V>(g.h1 + (size_t)i * W + c, u);
    if (g.h1_b) st_pack<V>(g.h1_b + (size_t)i * W + c, u);
    if (g.w2) {
      const Pack<V> w2 = early ? w2e : ld_pack<V>((const T*)g.w2 + c);
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

// Rows a workgroup convolves one after another, with the inputs of the last kRowTaps - 1 rows and the
// weights in registers.
constexpr int kRowBlock = 8;
constexpr int kRowTaps = 8;

// The input b steps before row r (of an entry with t rows before it in the batch).
template <int V>
__device__ __forceinline__ Pack<V> conv_input(const float* x, int64_t ldx, const float* state, int C, int taps, int r, int c,
                                              int b, int t, int pos, int slot) {
  if (b <= t) return ld_pack<V>(x + (size_t)(r - b) * ldx + c);
  if (pos - b >= 0) return ld_pack<V>(state + ((size_t)slot * (taps - 1) + (taps - 1 - (b - t))) * C + c);
  Pack<V> z;
#pragma unroll
  for (int e = 0; e < V; ++e) z.v[e] = 0.f;
  return z;
}

// out = x + conv(x): x's entry rows before r, then the sequence's state, then zeros.  A workgroup
// per (block of rows, 256 pieces of V channels).
template <typename T, int V>
__global__ __launch_bounds__(256) void conv_add_rows_kernel(
    const float* __restrict__ x, int64_t ldx, const T* __restrict__ w, const float* __restrict__ state,
    const int32_t* __restrict__ row_pos, const int32_t* __restrict__ row_slot, float* __restrict__ out,
    bf16_t* __restrict__ out_b, int64_t ldo, int n_rows, int C, int taps) {
  const int rb = blockIdx.x * kRowBlock, c = (blockIdx.y * 256 + threadIdx.x) * V;
  if (c >= C) return;
  const bool few = taps <= kRowTaps;
  Pack<V> cur[kRowBlock], wt[kRowTaps], win[kRowTaps];   // wt[b], win[b]: b steps back
#pragma unroll
  for (int u = 0; u < kRowBlock; ++u) cur[u] = ld_pack<V>(x + (size_t)(rb + u < n_rows ? rb + u : n_rows - 1) * ldx + c);
#pragma unroll
  for (int b = 0; b < kRowTaps; ++b)
    if (few && b < taps) wt[b] = ld_pack<V>(w + (size_t)(taps - 1 - b) * C + c);
  int prev = -1;
#pragma unroll
  for (int u = 0; u < kRowBlock; ++u) {
    const int r = rb + u;
    if (r >= n_rows) return;
    const int slot = row_slot[r];
    Pack<V> acc;
#pragma unroll
    for (int e = 0; e < V; ++e) acc.v[e] = 0.f;
    if (few) {
      if (slot != prev) {
        const int pos = row_pos[r], t = u == 0 ? rows_before(row_slot, r, taps) : 0;
#pragma unroll
        for (int b = 1; b < kRowTaps; ++b)
          if (b < taps) win[b] = conv_input<V>(x, ldx, state, C, taps, r, c, b, t, pos, slot);
      }
#pragma unroll
      for (int b = kRowTaps - 1; b >= 1; --b)
        if (b < taps) {
#pragma unroll
          for (int e = 0; e < V; ++e) acc.v[e] = fmaf(wt[b].v[e], win[b].v[e], acc.v[e]);
        }
#pragma unroll
      for (int e = 0; e < V; ++e) acc.v[e] = fmaf(wt[0].v[e], cur[u].v[e], acc.v[e]);
#pragma unroll
      for (int b = kRowTaps - 1; b >= 2; --b) win[b] = win[b - 1];
      win[1] = cur[u];
      prev = slot;
    } else {
      const int pos = row_pos[r], t = rows_before(row_slot, r, taps);
      for (int b = taps - 1; b >= 0; --b) {
        const Pack<V> in = conv_input<V>(x, ldx, state, C, taps, r, c, b, t, pos, slot);
        const Pack<V> wb = ld_pack<V>(w + (size_t)(taps - 1 - b) * C + c);
#pragma unroll
        for (int e = 0; e < V; ++e) acc.v[e] = fmaf(wb.v[e], in.v[e], acc.v[e]);
      }
    }
#pragma unroll
    for (int e = 0; e < V; ++e) acc.v[e] += cur[u].v[e];
    if (out) st_pack<V>(out + (size_t)r * ldo + c, acc);
    if (out_b) st_pack<V>(out_b + (size_t)r * ldo + c, acc);
  }
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
// the row's F values.  By a whole workgroup (whole waves; red: 3 floats a wave); pieces of V values,
// the first kPolyRegs of a thread held in registers between the sums and the result.
constexpr int kPolyRegs = 8;
template <typename T, int V>
__device__ __forceinline__ void poly_norm_pieces(const float* __restrict__ z, const T* __restrict__ bias,
                                                 const float* __restrict__ coef, float eps, int F,
                                                 float* __restrict__ out, bf16_t* __restrict__ out_b, float* red) {
  const int np = F / V, nthr = blockDim.x;
  auto piece = [&](int i) {
    Pack<V> v = ld_pack<V>(z + (size_t)i * V);
    if (bias) {
      const Pack<V> b = ld_pack<V>(bias + (size_t)i * V);
#pragma unroll
      for (int e = 0; e < V; ++e) v.v[e] += b.v[e];
    }
    return v;
  };
  float s1 = 0.f, s2 = 0.f, s3 = 0.f;
  auto add = [&](const Pack<V>& v) {
#pragma unroll
    for (int e = 0; e < V; ++e) {
      const float q = v.v[e] * v.v[e];
      s1 += q;
      s2 = fmaf(q, q, s2);
      s3 = fmaf(q * q, q, s3);
    }
  };
  Pack<V> keep[kPolyRegs];
#pragma unroll
  for (int u = 0; u < kPolyRegs; ++u)
    if (nthr * u < np) {   // (on a piece clamped into the row)
      const int i = threadIdx.x + nthr * u;
      keep[u] = piece(i < np ? i : np - 1);
    }
#pragma unroll
  for (int u = 0; u < kPolyRegs; ++u)
    if ((int)threadIdx.x + nthr * u < np) add(keep[u]);
  for (int i = threadIdx.x + nthr * kPolyRegs; i < np; i += nthr) add(piece(i));
  s1 = wave_sum(s1);
  s2 = wave_sum(s2);
  s3 = wave_sum(s3);
  const int wave = threadIdx.x >> 6, nw = nthr >> 6;
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
  auto write = [&](int i, const Pack<V>& v) {
    Pack<V> o;
#pragma unroll
    for (int e = 0; e < V; ++e) o.v[e] = fmaf(v.v[e], fmaf(v.v[e], fmaf(v.v[e], f3, f2), f1), f0);
    if (out) st_pack<V>(out + (size_t)i * V, o);
    if (out_b) st_pack<V>(out_b + (size_t)i * V, o);
  };
#pragma unroll
  for (int u = 0; u < kPolyRegs; ++u)
    if ((int)threadIdx.x + nthr * u < np) write(threadIdx.x + nthr * u, keep[u]);
  for (int i = threadIdx.x + nthr * kPolyRegs; i < np; i += nthr) write(i, piece(i));
}
template <typename T>
__device__ __forceinline__ void poly_norm_row(const float* __restrict__ z, const T* __restrict__ bias,
                                              const float* __restrict__ coef, float eps, int F,
                                              float* __restrict__ out, bf16_t* __restrict__ out_b, float* red) {
  const uintptr_t at = reinterpret_cast<uintptr_t>(z) | reinterpret_cast<uintptr_t>(out) |
                       (reinterpret_cast<uintptr_t>(bias) * (16 / (4 * sizeof(T)))) |
                       (reinterpret_cast<uintptr_t>(out_b) * 2);
  if (F % 4 == 0 && (at & 15) == 0) poly_norm_pieces<T, 4>(z, bias, coef, eps, F, out, out_b, red);
  else poly_norm_pieces<T, 1>(z, bias, coef, eps, F, out, out_b, red);
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
  const void* conv_w;      // [taps, C]
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
        acc = fmaf(ld_f(cw + (size_t)(taps - 1 - j) * g.C + ch0 + c), in, acc);
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

// The same for many rows: a wave takes its unit through kRowBlock rows one after another, weights and
// the last inputs in registers (NC channels per lane).  States are left to conv_tail_kernel.
template <typename T, int NC>
__global__ __launch_bounds__(256) void conv_prep_block_kernel(ConvPrepArgs g, int n_rows) {
  const int rb = blockIdx.x * kRowBlock, y = blockIdx.y;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int kind = y < g.q_wgs ? 0 : (y < g.q_wgs + g.kv_wgs ? 1 : 2);   // q, k, v
  const int unit = (kind == 0 ? y : (kind == 1 ? y - g.q_wgs : y - g.q_wgs - g.kv_wgs)) * kUnitWaves + wave;
  if (unit >= (kind == 0 ? g.H : g.G)) return;
  const int d = kind == 2 ? g.dv : g.dk, taps = g.taps;
  const int ch0 = (kind == 0 ? 0 : (kind == 1 ? g.H * g.dk : (g.H + g.G) * g.dk)) + unit * d;
  const T* bias = (const T*)g.bias;
  const T* nw = (const T*)(kind == 0 ? g.q_w : g.k_w);
  float cur[kRowBlock][NC], wt[kRowTaps][NC], win[kRowTaps][NC], b[NC], norm[NC];
  int ch[NC];
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    ch[k] = ch0 + (lane + 64 * k < d ? lane + 64 * k : d - 1);   // (clamped: results there are dropped)
    b[k] = bias ? ld_f(bias + ch[k]) : 0.f;
    norm[k] = kind < 2 ? ld_f(nw + ch[k] - ch0) : 1.f;
#pragma unroll
    for (int u = 0; u < kRowBlock; ++u) cur[u][k] = g.proj[(size_t)(rb + u < n_rows ? rb + u : n_rows - 1) * g.ld + ch[k]];
#pragma unroll
    for (int t = 0; t < kRowTaps; ++t)
      if (t < taps) wt[t][k] = ld_f((const T*)g.conv_w + (size_t)(taps - 1 - t) * g.C + ch[k]);
  }
  int prev = -1;
#pragma unroll
  for (int u = 0; u < kRowBlock; ++u) {
    const int r = rb + u;
    if (r >= n_rows) return;
    const int slot = g.row_slot[r], pos = g.row_pos[r];
    if (slot != prev) {
      const int t = u == 0 ? rows_before(g.row_slot, r, taps) : 0;
#pragma unroll
      for (int k = 0; k < NC; ++k)
#pragma unroll
        for (int s = 1; s < kRowTaps; ++s)
          if (s < taps) {
            if (s <= t) win[s][k] = g.proj[(size_t)(r - s) * g.ld + ch[k]] + b[k];
            else if (pos - s >= 0) win[s][k] = g.conv_state[((size_t)slot * (taps - 1) + (taps - 1 - (s - t))) * g.C + ch[k]];
            else win[s][k] = 0.f;
          }
    }
    prev = slot;
    float val[NC], ss = 0.f;
#pragma unroll
    for (int k = 0; k < NC; ++k) {
      const float in = cur[u][k] + b[k];
      float acc = 0.f;
#pragma unroll
      for (int s = kRowTaps - 1; s >= 1; --s)
        if (s < taps) acc = fmaf(wt[s][k], win[s][k], acc);
      acc = fmaf(wt[0][k], in, acc);
#pragma unroll
      for (int s = kRowTaps - 1; s >= 2; --s) win[s][k] = win[s - 1][k];
      win[1][k] = in;
      val[k] = lane + 64 * k < d ? acc : 0.f;
      ss = fmaf(val[k], val[k], ss);
    }
    if (kind < 2) {
      const float f = 1.f / sqrtf(wave_sum(ss) / (float)d + g.eps);
      const float temp = kind == 0 && g.temp_every > 0
                             ? 1.f + g.temp_coef * logf((float)((pos + 1) / g.temp_every) + 1.f) : 1.f;
#pragma unroll
      for (int k = 0; k < NC; ++k) val[k] = val[k] * f * norm[k] * temp;
    }
    if (kind == 0) {
      float* q = g.q_out + (size_t)r * g.H * g.dk + unit * d;
#pragma unroll
      for (int k = 0; k < NC; ++k)
        if (lane + 64 * k < d) q[lane + 64 * k] = val[k];
    } else {
      const int pg = g.block_tables[(size_t)slot * g.max_blocks + pos / g.page];
      T* dst = (T*)(kind == 1 ? g.k_cache : g.v_cache) + (((size_t)pg * g.G + unit) * g.page + pos % g.page) * d;
#pragma unroll
      for (int k = 0; k < NC; ++k)
        if (lane + 64 * k < d) st_f(dst + lane + 64 * k, val[k]);
    }
  }
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

// Scan and read-out of rows that are alone in their entries: a workgroup per (row, head), so that the
// head's norm needs no second launch.  A thread owns a strip of 16 key channels of one value column
// (CT columns at a time); the same sums in the same order as mlstm_scan_kernel.
template <typename T>
__global__ __launch_bounds__(1024) void mlstm_step_kernel(MlstmArgs a, MlstmPostArgs g, const int32_t* __restrict__ row_pos,
                                                          int CT, int NS) {
  extern __shared__ float lds[];
  __shared__ float red[48];
  const int r = blockIdx.y, h = blockIdx.x, H = a.H, dk = a.dk, dv = a.dv, tid = threadIdx.x;
  if (h == H) {
    poly_norm_row<T>(g.z + (size_t)r * g.ldz, (const T*)g.z_bias, g.coef, g.eps, g.F,
                     g.act ? g.act + (size_t)r * g.ldy : nullptr, g.act_b ? g.act_b + (size_t)r * g.ldy : nullptr, red);
    return;
  }
  float* qs = lds;                 // [NS*16]
  float* ks = qs + NS * kStrip;
  float* part = ks + NS * kStrip;  // [NS][CT]
  float* o = part + NS * CT;       // [dv]
  const int slot = g.row_slot[r], pos = row_pos[r], c = tid % CT, s = tid / CT, r0 = s * kStrip;
  const size_t at = (size_t)slot * H + h, row = (size_t)r * a.ld;
  const bool kept = pos > 0;
  float* st = a.S + at * dk * dv;
  float S[kStrip];
  auto load = [&](int col) {       // (clamped addresses; what lies outside is zeroed or dropped)
    const int cc = col < dv ? col : dv - 1;
#pragma unroll
    for (int i = 0; i < kStrip; ++i) {
      const int rr = r0 + i < dk ? r0 + i : dk - 1;
      const float v = st[(size_t)rr * dv + cc];
      S[i] = kept && r0 + i < dk ? v : 0.f;
    }
  };
  load(c);
  float n_old = 0.f;
  if (tid < NS * kStrip) {
    const int cc = tid < dk ? tid : dk - 1;
    const float q = a.q[row + (size_t)h * dk + cc] * a.q_scale, k = a.k[row + (size_t)h * dk + cc];
    const float n = a.nrm[at * dk + cc];
    qs[tid] = tid < dk ? q : 0.f;
    ks[tid] = tid < dk ? k : 0.f;
    n_old = kept ? n : 0.f;
  }
  const float zi = a.zi[row + h] + a.bi[h], zf = a.zf[row + h] + a.bf[h];
  const float li = a.cap * tanhf(zi / a.cap), lf = log_sigmoid_f(a.cap * tanhf(zf / a.cap));
  const float m0 = kept ? a.m[at] : 0.f, m = fmaxf(lf + m0, li);
  const float d = expf(lf + m0 - m), add = expf(li - m);
  __syncthreads();
  float nq = 0.f;
  if (tid < dk) {
    const float n = fmaf(d, n_old, ks[tid] * add);
    a.nrm[at * dk + tid] = n;
    nq = n * qs[tid];
  }
  if (tid == 0) a.m[at] = m;
  for (int c0 = 0; c0 < dv; c0 += CT) {
    const int col = c0 + c;
    if (c0 > 0) load(col);
    if (s < NS) {
      const float av = add * a.v[row + (size_t)h * dv + (col < dv ? col : dv - 1)];
      float acc = 0.f;
#pragma unroll
      for (int i = 0; i < kStrip; ++i) {
        S[i] = fmaf(d, S[i], ks[r0 + i] * av);
        acc = fmaf(S[i], qs[r0 + i], acc);
      }
      part[s * CT + c] = acc;
      if (col < dv) {
#pragma unroll
        for (int i = 0; i < kStrip; ++i)
          if (r0 + i < dk) st[(size_t)(r0 + i) * dv + col] = S[i];
      }
    }
    __syncthreads();
    if (tid < CT && c0 + tid < dv) {
      float sum = part[tid];
      for (int i = 1; i < NS; ++i) sum += part[i * CT + tid];
      o[c0 + tid] = sum;
    }
    __syncthreads();
  }
  nq = block_sum(nq, red);
  const float inv = 1.f / (fmaxf(fabsf(nq), expf(-m)) + 1e-6f);
  float ss = 0.f;
  for (int i = tid; i < dv; i += blockDim.x) ss = fmaf(o[i] * inv, o[i] * inv, ss);
  const float rstd = 1.f / sqrtf(block_sum(ss, red) / (float)dv + g.eps);
  for (int i = tid; i < dv; i += blockDim.x) {
    const int ch = h * dv + i;
    const float y = o[i] * inv * rstd * ld_f((const T*)g.w + ch) * sigmoid_f(g.gate[(size_t)r * g.ldg + ch]);
    if (g.y) g.y[(size_t)r * g.ldy + ch] = y;
    if (g.y_b) g.y_b[(size_t)r * g.ldy + ch] = (bf16_t)y;
  }
}

// ------------------------------------------------------------------ window attention on the matrix cores
// Many rows over bf16 caches.  A workgroup takes one kv head and a tile of query rows of one portion:
// wh query heads of the kv head x (4 / wh) groups of 16 rows, a pair of waves each, which share the
// tiles of keys that are staged in LDS (keys as rows, values transposed).  Two tiles of 64 keys are
// staged at a time; the waves of a pair take one each and put their sums together at the end.  A wave
// computes S^T = K Q^T, so that a query's scores sit in one column of the accumulator and are, as
// they are, the right operand of O^T = V^T P^T (the keys of an MFMA step in the order the
// accumulators hold them).  Queries and weights enter as the sum of two bf16 parts, keys and values
// are the cache's bf16 values: products carry 2^-17 of their operands, sums, softmax, cap and
// distance are f32.  The distance's logarithm is formed once per distinct distance of a tile.  Kept
// first tokens that lie before the window's first page come first, in stages of their own.
struct TiledAttnArgs {
  const float* q;
  int64_t ldq;
  const bf16_t* k_cache;
  const bf16_t* v_cache;
  const int32_t* block_tables;
  const int32_t* entries;
  const float* sinks;      // [H] or nullptr: one more term exp(sink) of the denominator
  const float* dist1;      // or nullptr
  const float* dist2;
  const float* gates;      // [rows, ldg] or nullptr: heads' outputs times sigmoid of it
  int64_t ldg;
  float* out;
  bf16_t* out_b;
  int64_t ldo;
  float scale, softcap;
  int n_entries, max_blocks, H, G, dk, dv, window, keep_first, wh, n_hgroups;
};
constexpr int kTileKeys = 64;
constexpr int kPage = 16;
constexpr float kLog2e = 1.4426950408889634f;

// The portion and the first row (inside it) of the n-th group of `per` rows over all portions.
__device__ __forceinline__ bool nth_group(const int32_t* entries, int n_entries, int per, int n, int* e, int* first) {
  int i = 0;
  for (; i < n_entries; ++i) {
    const int groups = (entries[4 * i + 2] + per - 1) / per;
    if (n < groups) break;
    n -= groups;
  }
  *e = i;
  *first = n * per;
  return i < n_entries;
}

template <int KS, int VT>
constexpr size_t tiled_attn_lds() {   // (the tiles' place also takes one wave group's results)
  const size_t tiles = 2 * ((size_t)kTileKeys * (32 * KS + 8) + (size_t)16 * VT * (kTileKeys + 4)) * sizeof(bf16_t);
  const size_t sums = (size_t)4 * SD_WAVE * (4 * VT + 2) * sizeof(float);
  return (tiles > sums ? tiles : sums) + 8 * 80 * sizeof(float);
}
template <int KS, int VT>   // heads of up to 32 * KS key and 16 * VT value channels
__global__ __launch_bounds__(512) void tiled_window_attn_kernel(TiledAttnArgs g) {
  constexpr int KLD = 32 * KS + 8, VLD = kTileKeys + 4, NV = VT / 4, kStage = 2 * kTileKeys, nthr = 512;
  extern __shared__ __attribute__((aligned(16))) char attn_lds[];
  bf16_t* ks = reinterpret_cast<bf16_t*>(attn_lds);            // [2][64][KLD]
  bf16_t* vs = ks + 2 * kTileKeys * KLD;                       // [2][16 * VT][VLD]
  float* sums = reinterpret_cast<float*>(attn_lds);            // [4 * VT + 2][4][64], at the end
  float* away = reinterpret_cast<float*>(attn_lds + tiled_attn_lds<KS, VT>() - 8 * 80 * sizeof(float)) + 80 * (threadIdx.x >> 6);
  const int tid = threadIdx.x, group = tid >> 8, wave = (tid >> 6) & 3, lane = tid & 63, col = lane & 15, quad = lane >> 4;
  const int kvh = blockIdx.y, hgroup = blockIdx.z, qh = g.H / g.G, dk = g.dk, dv = g.dv;
  const int n_sub = 4 / g.wh, tq = 16 * n_sub;
  int e, first;
  if (!nth_group(g.entries, g.n_entries, tq, blockIdx.x, &e, &first)) return;
  const int slot = g.entries[4 * e], row0 = g.entries[4 * e + 1], len = g.entries[4 * e + 2], pos0 = g.entries[4 * e + 3];
  const int hw = hgroup * g.wh + wave % g.wh, sub = first + 16 * (wave / g.wh);
  const int n_rows = len - sub < 16 ? len - sub : 16;        // this wave's rows (<= 0: none)
  const bool works = hw < qh && n_rows > 0;
  const int h = kvh * qh + (hw < qh ? hw : qh - 1);
  const int p = pos0 + sub + col;                            // this lane's query
  const int32_t* tbl = g.block_tables + (size_t)slot * g.max_blocks;
  const int last = pos0 + (len < first + tq ? len : first + tq) - 1;   // the workgroup's last position
  int base0 = pos0 + first - g.window + 1;                   // the window's first page
  base0 = base0 > 0 ? base0 & ~(kPage - 1) : 0;
  const int n_kept = g.keep_first < base0 ? g.keep_first : base0;   // kept tokens before it
  const int kept_stages = (n_kept + kStage - 1) / kStage, stages = kept_stages + (last - base0) / kStage + 1;
  auto stage_base = [&](int s) { return s < kept_stages ? s * kStage : base0 + (s - kept_stages) * kStage; };
  const float r1 = g.dist1 ? g.dist1[h] : 0.f, r2 = g.dist1 ? g.dist2[h] : 0.f;

  bf16x8 qa[KS], qb[KS];                                     // the query's two parts
  {
    const int r = row0 + (works ? sub + (col < n_rows ? col : n_rows - 1) : 0);
    const float* qr = g.q + (size_t)r * g.ldq + (size_t)h * dk;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      const int c = 32 * s + 8 * quad;
      float f[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) f[i] = 0.f;
      if (c < dk) {
        const f32x4 a = *reinterpret_cast<const f32x4*>(qr + c), b = *reinterpret_cast<const f32x4*>(qr + c + 4);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          f[i] = a[i] * g.scale;
          f[4 + i] = b[i] * g.scale;
        }
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        qa[s][i] = (bf16_t)f[i];
        qb[s][i] = (bf16_t)(f[i] - (float)qa[s][i]);
      }
    }
  }
  // a thread's pieces of the staged keys: KS of 8 channels; of the values: NV of 8 channels of two keys
  const u32x4 zero = {0, 0, 0, 0};
  u32x4 kr[KS], vr[NV][2];
  int kpg[KS], vpg[NV];
  auto pages = [&](int b0) {     // the pages of the keys from b0 on (clamped: rows behind `last` are zeroed)
#pragma unroll
    for (int i = 0; i < KS; ++i) {
      const int j = b0 + (tid + nthr * i) / (4 * KS);
      kpg[i] = tbl[(j < last ? j : last) / kPage];
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int j = b0 + 2 * ((tid + nthr * i) / (2 * VT));
      vpg[i] = tbl[(j < last ? j : last) / kPage];
    }
  };
  auto fetch = [&](int b0) {
#pragma unroll
    for (int i = 0; i < KS; ++i) {
      const int idx = tid + nthr * i, j = b0 + idx / (4 * KS), c = 8 * (idx % (4 * KS));
      kr[i] = zero;
      if (j <= last && c < dk)
        kr[i] = *reinterpret_cast<const u32x4*>(g.k_cache + (((size_t)kpg[i] * g.G + kvh) * kPage + j % kPage) * dk + c);
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int idx = tid + nthr * i, j = b0 + 2 * (idx / (2 * VT)), c = 8 * (idx % (2 * VT));
      const bf16_t* v = g.v_cache + (((size_t)vpg[i] * g.G + kvh) * kPage + j % kPage) * dv + c;
      vr[i][0] = vr[i][1] = zero;
      if (j <= last && c < dv) vr[i][0] = *reinterpret_cast<const u32x4*>(v);
      if (j + 1 <= last && c < dv) vr[i][1] = *reinterpret_cast<const u32x4*>(v + dv);
    }
  };
  f32x4 o[VT];
#pragma unroll
  for (int t = 0; t < VT; ++t) o[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  // (a sink opens the first wave group's running maximum and sum; a query's sum is spread over its four lanes)
  const bool sunk = g.sinks && group == 0;
  float m_run = sunk ? g.sinks[h] : -INFINITY, l_run = sunk && quad == 0 ? 1.f : 0.f;
  const float cap = g.softcap, cap_in = cap > 0.f ? 2.f * kLog2e / cap : 0.f;

  pages(stage_base(0));
  fetch(stage_base(0));
  pages(stage_base(1));
  for (int stage = 0; stage < stages; ++stage) {
    const int base = stage_base(stage);
    // (a stage of kept tokens holds no key of the window; in the window's stages kept tokens are seen too)
    const int key_end = stage < kept_stages ? n_kept : 0x7fffffff;
    __syncthreads();
#pragma unroll
    for (int i = 0; i < KS; ++i) {
      const int idx = tid + nthr * i;
      *reinterpret_cast<u32x4*>(ks + (idx / (4 * KS)) * KLD + 8 * (idx % (4 * KS))) = kr[i];
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int idx = tid + nthr * i, c = 8 * (idx % (2 * VT)), j = 2 * (idx / (2 * VT));
      const bf16x8 a = __builtin_bit_cast(bf16x8, vr[i][0]), b = __builtin_bit_cast(bf16x8, vr[i][1]);
      bf16_t* dst = vs + (j / kTileKeys) * 16 * VT * VLD + c * VLD + j % kTileKeys;
#pragma unroll
      for (int u = 0; u < 8; ++u) *reinterpret_cast<bf16x2*>(dst + u * VLD) = bf16x2{a[u], b[u]};
    }
    const int gbase = base + group * kTileKeys;              // this wave's tile
    if (g.dist1) {   // entry n: distance pos0 + sub - gbase - 63 + n
      const int d0 = pos0 + sub - gbase - (kTileKeys - 1);
      away[lane] = r1 * log1pf(r2 * (float)(d0 + lane > 0 ? d0 + lane : 0));
      if (lane < 16) away[64 + lane] = r1 * log1pf(r2 * (float)(d0 + 64 + lane > 0 ? d0 + 64 + lane : 0));
    }
    __syncthreads();
    if (stage + 1 < stages) {
      fetch(stage_base(stage + 1));
      pages(stage_base(stage + 2));
    }
    if (!works || gbase > pos0 + sub + n_rows - 1 || gbase >= key_end) continue;   // (keys behind this wave's last query)
    const bf16_t* kt = ks + group * kTileKeys * KLD;
    const bf16_t* vt = vs + group * 16 * VT * VLD;
    f32x4 sc[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) {
      sc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        const bf16x8 a = *reinterpret_cast<const bf16x8*>(kt + (16 * t + col) * KLD + 32 * s + 8 * quad);
        sc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, qa[s], sc[t], 0, 0, 0);
        sc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, qb[s], sc[t], 0, 0, 0);
      }
    }
    float mx = m_run;
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int kk = 16 * t + 4 * quad + i, d = p - (gbase + kk);
        float v = sc[t][i];
        // cap tanh(v / cap) = cap - 2 cap / (e^(2 v / cap) + 1)
        if (cap > 0.f) v = fmaf(-2.f * cap, __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(v * cap_in) + 1.f), cap);
        if (g.dist1) v -= away[col + kTileKeys - 1 - kk];
        const int j = gbase + kk;
        v = d >= 0 && (d < g.window || j < g.keep_first) && j < key_end ? v : -INFINITY;
        sc[t][i] = v;
        mx = fmaxf(mx, v);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 16, SD_WAVE));
    mx = fmaxf(mx, __shfl_xor(mx, 32, SD_WAVE));
    const float ref = mx == -INFINITY ? 0.f : mx;            // (no key seen yet)
    const float corr = __builtin_amdgcn_exp2f((m_run - ref) * kLog2e);
    m_run = mx;
    float sum = 0.f;
    bf16x8 pa[2], pb[2];
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float w = __builtin_amdgcn_exp2f((sc[t][i] - ref) * kLog2e);
        sum += w;
        const bf16_t a = (bf16_t)w;
        pa[t >> 1][4 * (t & 1) + i] = a;
        pb[t >> 1][4 * (t & 1) + i] = (bf16_t)(w - (float)a);
      }
    l_run = fmaf(l_run, corr, sum);
    if (__any(corr != 1.f)) {
#pragma unroll
      for (int t = 0; t < VT; ++t) o[t] *= corr;
    }
#pragma unroll
    for (int t = 0; t < VT; ++t)
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        const bf16_t* vrow = vt + (16 * t + col) * VLD + 32 * u + 4 * quad;
        const bf16x4 a0 = *reinterpret_cast<const bf16x4*>(vrow), a1 = *reinterpret_cast<const bf16x4*>(vrow + 16);
        const bf16x8 a = {a0[0], a0[1], a0[2], a0[3], a1[0], a1[1], a1[2], a1[3]};
        o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, pa[u], o[t], 0, 0, 0);
        o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, pb[u], o[t], 0, 0, 0);
      }
  }
  l_run += __shfl_xor(l_run, 16, SD_WAVE);
  l_run += __shfl_xor(l_run, 32, SD_WAVE);
  // the pair's sums: the second wave leaves its own, the first adds them
  __syncthreads();
  if (group == 1) {
    float* mine = sums + wave * SD_WAVE + lane;
#pragma unroll
    for (int t = 0; t < VT; ++t)
#pragma unroll
      for (int i = 0; i < 4; ++i) mine[(4 * t + i) * 4 * SD_WAVE] = o[t][i];
    mine[4 * VT * 4 * SD_WAVE] = m_run;
    mine[(4 * VT + 1) * 4 * SD_WAVE] = l_run;
  }
  __syncthreads();
  if (group == 1 || !works || col >= n_rows) return;
  const float* other = sums + wave * SD_WAVE + lane;
  const float m2 = other[4 * VT * 4 * SD_WAVE], m_all = fmaxf(m_run, m2);   // (one of them saw the query's own key)
  const float f1 = __builtin_amdgcn_exp2f((m_run - m_all) * kLog2e), f2 = __builtin_amdgcn_exp2f((m2 - m_all) * kLog2e);
#pragma unroll
  for (int t = 0; t < VT; ++t)
#pragma unroll
    for (int i = 0; i < 4; ++i) o[t][i] = fmaf(o[t][i], f1, other[(4 * t + i) * 4 * SD_WAVE] * f2);
  float inv = 1.f / fmaf(l_run, f1, other[(4 * VT + 1) * 4 * SD_WAVE] * f2);
  if (g.gates) inv *= sigmoid_f(g.gates[(size_t)(row0 + sub + col) * g.ldg + h]);
  const size_t at = (size_t)(row0 + sub + col) * g.ldo + (size_t)h * dv;
  const bool quads = g.ldo % 4 == 0;
#pragma unroll
  for (int t = 0; t < VT; ++t) {
    const int c = 16 * t + 4 * quad;
    if (c >= dv) continue;
    const Pack<4> v = {{o[t][0] * inv, o[t][1] * inv, o[t][2] * inv, o[t][3] * inv}};
    if (quads) {
      if (g.out) st_pack<4>(g.out + at + c, v);
      if (g.out_b) st_pack<4>(g.out_b + at + c, v);
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        if (g.out) g.out[at + c + i] = v.v[i];
        if (g.out_b) g.out_b[at + c + i] = (bf16_t)v.v[i];
      }
    }
  }
}

// ------------------------------------------------------------------ the matrix memory in chunks
// The recurrence of mlstm_scan_kernel over chunks of 64 tokens, on the f32 matrix instruction (no
// reduced precision).  With D(t, s) the sum of the log forget gates of s+1 .. t and b_t = D(t, -1):
//   num_t = e^(b_t + m0 - m_t) q_t S0 + sum_{s <= t} e^(D(t, s) + i_s - m_t) (q_t . k_s) v_s,
// S0, m0 the memory and its running maximum at the chunk's start.  Three launches: every chunk's own
// sum of e^(D(63, s) + i_s - mu) k_s v_s^T with a maximum mu of its own (chunk_sums), the memories at
// the chunks' starts (chunk_carry, chunk after chunk), the tokens' results (chunk_reads).  A maximum
// only scales numbers, so mu and m_t need not be the ones another cut of the tokens would give.
struct MlstmChunkArgs {
  MlstmArgs a;
  int n_entries;
  float* cs;               // [chunks, H, dk, dv]: own sums, then the memory at the chunk's start
  float* cn;               // [chunks, H, dk]: the same of k alone
  float* sc;               // [chunks, H, 4]: b of the last token, mu, m at the start, m at the end
};
constexpr int kChunk = 64;

// log gates of the chunk's token `lane` (a token behind the chunk's end adds nothing)
__device__ __forceinline__ void chunk_gates(const MlstmArgs& a, int row, int h, bool in, float* li, float* lf) {
  const float zi = a.zi[(size_t)row * a.ld + h] + a.bi[h], zf = a.zf[(size_t)row * a.ld + h] + a.bf[h];
  *li = in ? a.cap * tanhf(zi / a.cap) : -INFINITY;
  *lf = in ? log_sigmoid_f(a.cap * tanhf(zf / a.cap)) : 0.f;
}

typedef __attribute__((ext_vector_type(16))) float acc32_t;
// row of register i of a 32x32 accumulator
__device__ __forceinline__ int acc_row(int i, int half) { return 8 * (i >> 2) + 4 * half + (i & 3); }

constexpr int kChunkCols = 128;   // value columns per workgroup
// 64 rows of up to COLS columns on their way from memory to LDS, V columns a piece: all of a thread's
// pieces are asked for at once (on addresses clamped into the valid part), then stored.
template <int COLS, int V>
struct ChunkRows {
  static constexpr int N = kChunk * COLS / V / 256;
  Pack<V> v[N];
  __device__ __forceinline__ void load(const float* src, int64_t ld, int rows, int cols) {
#pragma unroll
    for (int u = 0; u < N; ++u) {
      const int idx = threadIdx.x + 256 * u, t = idx / (COLS / V), c = idx % (COLS / V) * V;
      v[u] = ld_pack<V>(src + (size_t)(t < rows ? t : rows - 1) * ld + (c < cols ? c : cols - V));
    }
  }
  // times wt[row] (or f where wt is nullptr)
  __device__ __forceinline__ void store(float* dst, int ldd, int rows, int cols, const float* wt, float f) {
#pragma unroll
    for (int u = 0; u < N; ++u) {
      const int idx = threadIdx.x + 256 * u, t = idx / (COLS / V), c = idx % (COLS / V) * V;
      const float w = t < rows && c < cols ? (wt ? wt[t] : f) : 0.f;
#pragma unroll
      for (int e = 0; e < V; ++e) dst[t * ldd + c + e] = w == 0.f ? 0.f : v[u].v[e] * w;
    }
  }
};

template <int DKP, int V>   // keys of up to DKP channels
__global__ __launch_bounds__(256) void mlstm_chunk_sums_kernel(MlstmChunkArgs g) {
  extern __shared__ float lds[];
  const MlstmArgs& a = g.a;
  const int dk = a.dk, dv = a.dv, H = a.H;
  constexpr int nkt = DKP / 32;
  float* ks = lds;                   // [64][DKP], times the token's weight
  float* vs = ks + kChunk * DKP;     // [64][128]
  float* wt = vs + kChunk * kChunkCols;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, l31 = lane & 31, half = lane >> 5;
  const int h = blockIdx.y, c0 = blockIdx.z * kChunkCols, cols = dv - c0 < kChunkCols ? dv - c0 : kChunkCols;
  int e, first;
  if (!nth_group(a.entries, g.n_entries, kChunk, blockIdx.x, &e, &first)) return;
  const int row0 = a.entries[4 * e + 1] + first, left = a.entries[4 * e + 2] - first, nt = left < kChunk ? left : kChunk;
  const size_t at = (size_t)blockIdx.x * H + h;
  ChunkRows<DKP, V> kr;
  ChunkRows<kChunkCols, V> vr;
  kr.load(a.k + (size_t)row0 * a.ld + (size_t)h * dk, a.ld, nt, dk);
  vr.load(a.v + (size_t)row0 * a.ld + (size_t)h * dv + c0, a.ld, nt, cols);
  if (wave == 0) {
    float li, lf;
    chunk_gates(a, row0 + (lane < nt ? lane : nt - 1), h, lane < nt, &li, &lf);
    float d = __shfl_down(lf, 1, SD_WAVE);        // sum of the gates behind this token
    if (lane == 63) d = 0.f;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float n = __shfl_down(d, o, SD_WAVE);
      if (lane + o < 64) d += n;
    }
    const float mu = wave_max(d + li);
    wt[lane] = expf(d + li - mu);
    if (lane == 0 && blockIdx.z == 0) {
      g.sc[at * 4] = d + lf;
      g.sc[at * 4 + 1] = mu;
    }
  }
  vr.store(vs, kChunkCols, nt, cols, nullptr, 1.f);
  __syncthreads();
  kr.store(ks, DKP, nt, dk, wt, 0.f);
  __syncthreads();
  const int nct = (cols + 31) / 32;
  float* cs = g.cs + at * dk * dv + c0;
  for (int p = wave; p < nkt * nct; p += 4) {
    const int kt = p % nkt, ct = p / nkt;
    acc32_t acc;
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[i] = 0.f;
    const float* ka = ks + half * DKP + 32 * kt + l31;
    const float* vb = vs + half * kChunkCols + 32 * ct + l31;
#pragma unroll
    for (int s = 0; s < kChunk; s += 2)
      acc = __builtin_amdgcn_mfma_f32_32x32x2f32(ka[s * DKP], vb[s * kChunkCols], acc, 0, 0, 0);
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int r = 32 * kt + acc_row(i, half);
      if (r < dk && 32 * ct + l31 < cols) cs[(size_t)r * dv + 32 * ct + l31] = acc[i];
    }
  }
  if (blockIdx.z == 0 && tid < dk) {
    float n = 0.f;
#pragma unroll 16
    for (int s = 0; s < kChunk; ++s) n += ks[s * DKP + tid];
    g.cn[at * dk + tid] = n;
  }
}

// One element of a head's memory (or normalizer) through the chunks of its portion.
__global__ __launch_bounds__(256) void mlstm_chunk_carry_kernel(MlstmChunkArgs g) {
  const MlstmArgs& a = g.a;
  const int dk = a.dk, dv = a.dv, H = a.H, h = blockIdx.y, e = blockIdx.z;
  const int x = blockIdx.x * 256 + threadIdx.x;
  const int slot = a.entries[4 * e], len = a.entries[4 * e + 2], pos0 = a.entries[4 * e + 3];
  int c0 = 0;
  for (int i = 0; i < e; ++i) c0 += (a.entries[4 * i + 2] + kChunk - 1) / kChunk;
  const int nc = (len + kChunk - 1) / kChunk;
  const bool is_n = x >= dk * dv;
  if (x >= dk * dv + dk) return;
  float* st = is_n ? a.nrm + ((size_t)slot * H + h) * dk + (x - dk * dv) : a.S + ((size_t)slot * H + h) * dk * dv + x;
  float* own = is_n ? g.cn + ((size_t)c0 * H + h) * dk + (x - dk * dv) : g.cs + ((size_t)c0 * H + h) * dk * dv + x;
  const size_t step = is_n ? (size_t)H * dk : (size_t)H * dk * dv;
  float* sc = g.sc + ((size_t)c0 * H + h) * 4;
  float val = pos0 > 0 ? *st : 0.f, m = pos0 > 0 ? a.m[(size_t)slot * H + h] : 0.f;
  constexpr int U = 8;
  for (int i = 0; i < nc; i += U) {
    float v[U], b[U], mu[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = i + u < nc ? i + u : nc - 1;
      v[u] = own[c * step];
      b[u] = sc[(size_t)c * H * 4];
      mu[u] = sc[(size_t)c * H * 4 + 1];
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (i + u >= nc) break;
      const float m_new = fmaxf(b[u] + m, mu[u]);
      own[(i + u) * step] = val;
      val = fmaf(expf(b[u] + m - m_new), val, expf(mu[u] - m_new) * v[u]);
      if (x == 0) {
        sc[(size_t)(i + u) * H * 4 + 2] = m;
        sc[(size_t)(i + u) * H * 4 + 3] = m_new;
      }
      m = m_new;
    }
  }
  *st = val;
}

template <int DKP, int V>
__global__ __launch_bounds__(256) void mlstm_chunk_reads_kernel(MlstmChunkArgs g) {
  extern __shared__ float lds[];
  const MlstmArgs& a = g.a;
  const int dk = a.dk, dv = a.dv, H = a.H;
  constexpr int ldk = DKP + 1, kLdA = kChunk + 1, kSteps = DKP / 2;
  float* qs = lds;                     // [64][ldk]
  float* ks = qs + kChunk * ldk;       // [64][ldk]
  float* vs = ks + kChunk * ldk;       // [64][128]
  float* as = vs + kChunk * kChunkCols;  // [64][65] weighted scores
  float* lis = as + kChunk * kLdA;     // [64] each
  float* lfs = lis + kChunk;
  float* ms = lfs + kChunk;
  float* carry = ms + kChunk;
  float* ns = carry + kChunk;          // [DKP]
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, l31 = lane & 31, half = lane >> 5;
  const int h = blockIdx.y, c0 = blockIdx.z * kChunkCols, cols = dv - c0 < kChunkCols ? dv - c0 : kChunkCols;
  int e, first;
  if (!nth_group(a.entries, g.n_entries, kChunk, blockIdx.x, &e, &first)) return;
  const int row0 = a.entries[4 * e + 1] + first, left = a.entries[4 * e + 2] - first, nt = left < kChunk ? left : kChunk;
  const size_t at = (size_t)blockIdx.x * H + h;
  ChunkRows<DKP, V> qr, kr;
  ChunkRows<kChunkCols, V> vr;
  qr.load(a.q + (size_t)row0 * a.ld + (size_t)h * dk, a.ld, nt, dk);
  kr.load(a.k + (size_t)row0 * a.ld + (size_t)h * dk, a.ld, nt, dk);
  vr.load(a.v + (size_t)row0 * a.ld + (size_t)h * dv + c0, a.ld, nt, cols);
  // the memory at the chunk's start: this wave's 32 columns, rows 2 j + half
  const int wcol = 32 * wave + l31;
  const bool col_in = wcol < cols;
  float S[kSteps];
  {
    const float* s0 = g.cs + at * dk * dv + c0 + (col_in ? wcol : 0);
#pragma unroll
    for (int j = 0; j < kSteps; ++j) {
      const int r = 2 * j + half;
      const float v = s0[(size_t)(r < dk ? r : dk - 1) * dv];
      S[j] = r < dk && col_in ? v : 0.f;
    }
  }
  if (wave == 0) {
    float li, lf;
    chunk_gates(a, row0 + (lane < nt ? lane : nt - 1), h, lane < nt, &li, &lf);
    const float m0 = g.sc[at * 4 + 2], m1 = g.sc[at * 4 + 3];
    float F = lf, I = li;              // (F, I): m = max(F + m0, I), composed over the tokens so far
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float fp = __shfl_up(F, o, SD_WAVE), ip = __shfl_up(I, o, SD_WAVE);
      if (lane >= o) {
        I = fmaxf(ip + F, I);
        F += fp;
      }
    }
    float m = fmaxf(F + m0, I);
    if (lane == nt - 1) m = m1;        // the maximum the carried memory was scaled with
    lis[lane] = li;
    lfs[lane] = lf;
    ms[lane] = m;
    carry[lane] = expf(F + m0 - m);
    if (blockIdx.z == 0 && lane < nt) a.m_rows[(size_t)(row0 + lane) * H + h] = m;
  } else {
    for (int c = tid - 64; c < DKP; c += 192) ns[c] = c < dk ? g.cn[at * dk + c] : 0.f;
  }
  qr.store(qs, ldk, nt, dk, nullptr, a.q_scale);
  kr.store(ks, ldk, nt, dk, nullptr, 1.f);
  vr.store(vs, kChunkCols, nt, cols, nullptr, 1.f);
  __syncthreads();
  {
    // the tokens' weights: lane s, sixteen tokens t per wave; D(t, s) is summed from s on, so that a
    // long stretch of forgetting before s costs nothing of its precision
    const float li = lis[lane];
    float d = 0.f;
    const int t0 = 16 * wave;
#pragma unroll 16
    for (int t = 0; t < t0; ++t) d += t > lane ? lfs[t] : 0.f;
#pragma unroll
    for (int u = 0; u < 16; ++u) {
      const int t = t0 + u;
      d += t > lane ? lfs[t] : 0.f;
      as[t * kLdA + lane] = t >= lane ? expf(d + li - ms[t]) : 0.f;
    }
  }
  acc32_t acc[2];
  {
    const int tt = wave >> 1, ss = wave & 1;    // q k^T, a 32 x 32 part per wave
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[0][i] = 0.f;
    const float* qa = qs + (32 * tt + l31) * ldk + half;
    const float* kb = ks + (32 * ss + l31) * ldk + half;
    if (tt >= ss) {
#pragma unroll
      for (int c = 0; c < DKP; c += 2) acc[0] = __builtin_amdgcn_mfma_f32_32x32x2f32(qa[c], kb[c], acc[0], 0, 0, 0);
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 16; ++i) as[(32 * tt + acc_row(i, half)) * kLdA + 32 * ss + l31] *= acc[0][i];
  }
#pragma unroll
  for (int u = 0; u < 2; ++u)
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[u][i] = 0.f;
#pragma unroll
  for (int j = 0; j < kSteps; ++j)
#pragma unroll
    for (int u = 0; u < 2; ++u)
      acc[u] = __builtin_amdgcn_mfma_f32_32x32x2f32(qs[(32 * u + l31) * ldk + 2 * j + half], S[j], acc[u], 0, 0, 0);
#pragma unroll
  for (int u = 0; u < 2; ++u)
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[u][i] *= carry[32 * u + acc_row(i, half)];
  __syncthreads();
  // (the first 32 tokens see nothing of the later ones)
#pragma unroll
  for (int s = 0; s < 32; s += 2) {
    const float b = vs[(s + half) * kChunkCols + wcol];
    acc[0] = __builtin_amdgcn_mfma_f32_32x32x2f32(as[l31 * kLdA + s + half], b, acc[0], 0, 0, 0);
    acc[1] = __builtin_amdgcn_mfma_f32_32x32x2f32(as[(32 + l31) * kLdA + s + half], b, acc[1], 0, 0, 0);
  }
#pragma unroll
  for (int s = 32; s < 64; s += 2)
    acc[1] = __builtin_amdgcn_mfma_f32_32x32x2f32(as[(32 + l31) * kLdA + s + half], vs[(s + half) * kChunkCols + wcol], acc[1],
                                                  0, 0, 0);
  if (col_in) {
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int t = 32 * u + acc_row(i, half);
        if (t < nt) a.num[((size_t)(row0 + t) * H + h) * (dv + 1) + c0 + wcol] = acc[u][i];
      }
  }
  if (blockIdx.z == 0) {   // n . q, four threads a token
    const int t = tid >> 2, part = tid & 3;
    float n = 0.f, o = 0.f;
    for (int c = part; c < DKP; c += 4) n = fmaf(qs[t * ldk + c], ns[c], n);
    for (int s = part; s < kChunk; s += 4) o += as[t * kLdA + s];
    n = fmaf(n, carry[t], o);
    n += __shfl_xor(n, 1, SD_WAVE);
    n += __shfl_xor(n, 2, SD_WAVE);
    if (part == 0 && t < nt) a.num[((size_t)(row0 + t) * H + h) * (dv + 1) + dv] = n;
  }
}

template <int DKP, int V>
hipError_t launch_chunks(const MlstmChunkArgs& c, size_t nc, hipStream_t st) {
  static std::once_flag once;
  static hipError_t err = hipSuccess;
  std::call_once(once, [] {
    err = hipFuncSetAttribute(reinterpret_cast<const void*>(mlstm_chunk_sums_kernel<DKP, V>),
                              hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    if (err == hipSuccess)
      err = hipFuncSetAttribute(reinterpret_cast<const void*>(mlstm_chunk_reads_kernel<DKP, V>),
                                hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
  });
  if (err != hipSuccess) return err;
  const int dk = c.a.dk, dv = c.a.dv, H = c.a.H;
  const dim3 grid((unsigned)nc, H, (dv + kChunkCols - 1) / kChunkCols);
  const size_t lds1 = sizeof(float) * ((size_t)kChunk * DKP + (size_t)kChunk * kChunkCols + kChunk);
  const size_t lds2 = sizeof(float) * (2 * kChunk * (DKP + 1) + (size_t)kChunk * kChunkCols + kChunk * (kChunk + 1) +
                                       4 * kChunk + DKP);
  mlstm_chunk_sums_kernel<DKP, V><<<grid, 256, lds1, st>>>(c);
  mlstm_chunk_carry_kernel<<<dim3((dk * dv + dk + 255) / 256, H, c.n_entries), 256, 0, st>>>(c);
  mlstm_chunk_reads_kernel<DKP, V><<<grid, 256, lds2, st>>>(c);
  return hipGetLastError();
}
// chunks that n_entries portions of n_rows rows in all may have
inline size_t max_chunks(int n_rows, int n_entries) { return (size_t)n_rows / kChunk + n_entries; }

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
  dim3 grid((n_rows + kRowBlock - 1) / kRowBlock, ((quad ? C / 4 : C) + 255) / 256);
#define SD_GO(T, V) conv_add_rows_kernel<T, V><<<grid, 256, 0, st>>>(x, ldx, (const T*)w, conv_state, row_pos, row_slot, out, (bf16_t*)out_bf16, ldo, n_rows, C, taps)
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
  hipStream_t st = (hipStream_t)stream;
  const int units = g.q_wgs + (shared ? 0 : 2 * g.kv_wgs);
  if (!g.single && n_rows > 2 * kRowBlock && taps <= kRowTaps) {
    if (act)
      if (const int rc = sd_poly_norm_rows(act->z, act->ldz, act->bias, w_f32, act->coef, eps, act->out, act->out_bf16,
                                           act->ldo, n_rows, act->n, stream))
        return rc;
    const dim3 gb((n_rows + kRowBlock - 1) / kRowBlock, units);
    const int d = dk > dv ? dk : dv;
#define SD_GO(T)                                                              \
  do {                                                                        \
    if (d <= 64) conv_prep_block_kernel<T, 1><<<gb, 256, 0, st>>>(g, n_rows);        \
    else if (d <= 128) conv_prep_block_kernel<T, 2><<<gb, 256, 0, st>>>(g, n_rows);  \
    else if (d <= 256) conv_prep_block_kernel<T, 4><<<gb, 256, 0, st>>>(g, n_rows);  \
    else conv_prep_block_kernel<T, 8><<<gb, 256, 0, st>>>(g, n_rows);                \
  } while (0)
    if (w_f32) SD_GO(float);
    else SD_GO(bf16_t);
#undef SD_GO
    SD_CHECK_LAUNCH("sd_conv_attn_prep");
    return sd_conv_tail(proj, ld, bias, w_f32, conv_state, entries, n_entries, g.C, taps, stream);
  }
  dim3 grid(n_rows, units + (act ? 1 : 0));
  if (w_f32) conv_prep_kernel<float><<<grid, 256, 0, st>>>(g);
  else conv_prep_kernel<bf16_t><<<grid, 256, 0, st>>>(g);
  SD_CHECK_LAUNCH("sd_conv_attn_prep");
  if (g.single) return SD_OK;
  return sd_conv_tail(proj, ld, bias, w_f32, conv_state, entries, n_entries, g.C, taps, stream);
}

extern "C" size_t sd_mlstm_scratch_bytes(int n_rows, int n_entries, int H, int dk, int dv) {
  // (a few rows beyond one per portion do not fill chunks: token by token is as fast)
  if (n_rows < 1 || n_entries < 1 || n_rows - n_entries < kChunk / 2 || H < 1 || dk < 1 || dk > 128 || dv < 1) return 0;
  return sizeof(float) * max_chunks(n_rows, n_entries) * H * ((size_t)dk * dv + dk + 4);
}

extern "C" int sd_mlstm_scan(const float* q, const float* k, const float* v, const float* zi, const float* zf,
                             int64_t ld, const float* bi, const float* bf, float cap, float q_scale, float* S,
                             float* n_state, const float* m_state, const int32_t* entries, int n_entries, int n_rows,
                             float* num, float* m_rows, int H, int dk, int dv, void* scratch, size_t scratch_bytes,
                             sd_stream_t stream) {
  SD_REQUIRE(q && k && v && zi && zf && bi && bf && S && n_state && m_state && entries && num && m_rows &&
                 n_entries >= 1 && n_rows >= n_entries && H >= 1 && dv >= 1 && cap > 0.f,
             SD_ERR_INVALID, "sd_mlstm_scan: bad argument");
  SD_REQUIRE(dk >= 1 && dk <= 256, SD_ERR_UNSUPPORTED, "sd_mlstm_scan: key size %d outside 1..256", dk);
  hipStream_t st = (hipStream_t)stream;
  MlstmArgs g{q, k, v, zi, zf, ld, bi, bf, cap, q_scale, S, n_state, const_cast<float*>(m_state), entries, num, m_rows, H, dk, dv};
  const size_t need = sd_mlstm_scratch_bytes(n_rows, n_entries, H, dk, dv);
  if (need > 0 && scratch && scratch_bytes >= need && sd_aligned16(scratch)) {
    const size_t nc = max_chunks(n_rows, n_entries);
    MlstmChunkArgs c{g, n_entries, (float*)scratch, nullptr, nullptr};
    c.cn = c.cs + nc * H * dk * dv;
    c.sc = c.cn + nc * H * dk;
    // (four columns a piece where every row's pieces are 16-byte aligned)
    const bool quad = ld % 4 == 0 && dk % 4 == 0 && dv % 4 == 0 && sd_aligned16(q) && sd_aligned16(k) && sd_aligned16(v);
    hipError_t err;
    if (dk <= 32) err = quad ? launch_chunks<32, 4>(c, nc, st) : launch_chunks<32, 1>(c, nc, st);
    else if (dk <= 64) err = quad ? launch_chunks<64, 4>(c, nc, st) : launch_chunks<64, 1>(c, nc, st);
    else err = quad ? launch_chunks<128, 4>(c, nc, st) : launch_chunks<128, 1>(c, nc, st);
    SD_REQUIRE(err == hipSuccess, SD_ERR_HIP, "sd_mlstm_scan: launch failed: %s", hipGetErrorString(err));
    return SD_OK;
  }
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
  mlstm_scan_kernel<<<dim3((cols + CT - 1) / CT, H, n_entries), CT * NS, lds, st>>>(g, CT, NS, CH);
  SD_CHECK_LAUNCH("sd_mlstm_scan");
  return SD_OK;
}

int sd_tiled_window_attention_(const float* q, int64_t ldq, const void* k_cache, const void* v_cache,
                               const int32_t* block_tables, int max_blocks, int page, int n_rows, int H,
                               int G, int dk, int dv, int window, int keep_first, float scale, float softcap,
                               const float* sinks, const float* dist1, const float* dist2, const float* gates,
                               int64_t ldg, const int32_t* entries, int n_entries, float* out, void* out_bf16,
                               int64_t ldo, sd_stream_t stream) {
  if (page != kPage || dk % 8 || dv % 8 || dk > 128 || dv > 128 || ldq % 4 || !sd_aligned16(q) || !sd_aligned16(k_cache) ||
      !sd_aligned16(v_cache) || !(ldo % 4 || (sd_aligned16(out) && sd_aligned16(out_bf16))))
    return SD_ERR_UNSUPPORTED;
  const int qh = H / G;
  TiledAttnArgs g{q, ldq, (const bf16_t*)k_cache, (const bf16_t*)v_cache, block_tables, entries, sinks, dist1, dist2,
                  gates, ldg, out, (bf16_t*)out_bf16, ldo, scale, softcap, n_entries, max_blocks, H, G, dk, dv, window,
                  keep_first, 0, 0};
  g.wh = qh >= 4 ? 4 : (qh >= 2 ? 2 : 1);
  g.n_hgroups = (qh + g.wh - 1) / g.wh;
  const int tq = 16 * (4 / g.wh);
  dim3 grid(n_rows / tq + n_entries, G, g.n_hgroups);
  hipStream_t st = (hipStream_t)stream;
#define SD_GO(KS, VT)                                                                                                    \
  do {                                                                                                                   \
    static std::once_flag once;                                                                                          \
    static hipError_t err = hipSuccess;                                                                                  \
    std::call_once(once, [] {                                                                                            \
      err = hipFuncSetAttribute(reinterpret_cast<const void*>(tiled_window_attn_kernel<KS, VT>),                         \
                                hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);                                 \
    });                                                                                                                  \
    SD_REQUIRE(err == hipSuccess, SD_ERR_HIP, "sd_distance_softmax_attention: hipFuncSetAttribute failed: %s",           \
               hipGetErrorString(err));                                                                                  \
    tiled_window_attn_kernel<KS, VT><<<grid, 512, tiled_attn_lds<KS, VT>(), st>>>(g);                                    \
  } while (0)
  if (dk <= 64 && dv <= 64) SD_GO(2, 4);
  else if (dk <= 64) SD_GO(2, 8);
  else if (dv <= 64) SD_GO(4, 4);
  else SD_GO(4, 8);
#undef SD_GO
  SD_CHECK_LAUNCH("sd_distance_softmax_attention (tiled)");
  return SD_OK;
}

extern "C" int sd_mlstm_step(const float* q, const float* k, const float* v, const float* zi, const float* zf,
                             int64_t ld, const float* bi, const float* bf, float cap, float q_scale, float* S,
                             float* n_state, float* m_state, const int32_t* row_pos, const int32_t* row_slot,
                             const float* gate, const void* w, int w_f32, float eps, float* y, void* y_bf16,
                             int64_t ldy, int n_rows, int H, int dk, int dv, const sd_poly_norm* act,
                             sd_stream_t stream) {
  SD_REQUIRE(q && k && v && zi && zf && bi && bf && S && n_state && m_state && row_pos && row_slot && gate && w &&
                 (y || y_bf16) && n_rows >= 1 && H >= 1 && dv >= 1 && cap > 0.f && ldy >= (int64_t)H * dv,
             SD_ERR_INVALID, "sd_mlstm_step: bad argument");
  SD_REQUIRE(dk >= 1 && dk <= 256 && dv <= 4096, SD_ERR_UNSUPPORTED, "sd_mlstm_step: key size %d / value size %d", dk, dv);
  SD_REQUIRE(!act || (act->z && act->coef && (act->out || act->out_bf16) && act->n >= 1 && act->ldz >= act->n && act->ldo == ldy),
             SD_ERR_INVALID, "sd_mlstm_step: bad activation");
  MlstmArgs a{q, k, v, zi, zf, ld, bi, bf, cap, q_scale, S, n_state, m_state, nullptr, nullptr, nullptr, H, dk, dv};
  MlstmPostArgs g{};
  g.row_slot = row_slot; g.gate = gate; g.ldg = ld; g.w = w; g.eps = eps; g.y = y; g.y_b = (bf16_t*)y_bf16; g.ldy = ldy;
  g.H = H; g.dv = dv;
  if (act) {
    g.z = act->z; g.ldz = act->ldz; g.z_bias = act->bias; g.coef = act->coef; g.act = act->out;
    g.act_b = (bf16_t*)act->out_bf16; g.F = act->n;
  }
  const int NS = (dk + kStrip - 1) / kStrip;
  int CT = 1024 / NS / 64 * 64;
  if (CT > (dv + 63) / 64 * 64) CT = (dv + 63) / 64 * 64;
  int nthr = CT * NS;
  if (nthr < 256) nthr = 256;
  const size_t lds = sizeof(float) * ((size_t)2 * NS * kStrip + (size_t)NS * CT + dv);
  hipStream_t st = (hipStream_t)stream;
  dim3 grid(H + (act ? 1 : 0), n_rows);
  if (w_f32) mlstm_step_kernel<float><<<grid, nthr, lds, st>>>(a, g, row_pos, CT, NS);
  else mlstm_step_kernel<bf16_t><<<grid, nthr, lds, st>>>(a, g, row_pos, CT, NS);
  SD_CHECK_LAUNCH("sd_mlstm_step");
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
