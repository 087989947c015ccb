// Mechanisms of decoders that keep several copies of the residual (streams): the update of all
// streams with the norm of the next sublayer's input, the preparation of attention inputs with
// biases and a norm per head, and linear attention with a decay per key channel: the decays from a
// low-rank pair of matrices, prompts in chunks on the f32 matrix instruction, single decoded tokens
// in one launch with their read-out.
//
// Arithmetic as in sd_seqmix.hip: activations are f32 buffers; streams, norms, decays and states are
// f32 always; with bf16 weights the operands of matrix products are rounded to bf16 where they are
// produced and the cache holds bf16.
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
  return fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
}

// Sums of two numbers over a workgroup of up to 16 waves (butterfly inside each wave, then the waves in
// order); red: 32 floats.
struct Two { float a, b; };
__device__ __forceinline__ Two block_sum2(float a, float b, float* red) {
  a = wave_sum(a);
  b = wave_sum(b);
  const int wave = threadIdx.x >> 6, n_waves = (blockDim.x + 63) >> 6;
  __syncthreads();
  if ((threadIdx.x & 63) == 0) {
    red[wave] = a;
    red[16 + wave] = b;
  }
  __syncthreads();
  Two s = {red[0], red[16]};
  for (int w = 1; w < n_waves; ++w) {
    s.a += red[w];
    s.b += red[16 + w];
  }
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

// ------------------------------------------------------------------ the streams
// A workgroup per row, in three steps: the sublayer's result y (its norms' sums), the streams' update and
// the next sublayer's input u, u's norm.  A thread's first piece of V columns stays in registers from
// step to step (the streams' loads are asked for before the first sum is formed); further pieces are
// read again, u waits in LDS.  SM: streams at most.
template <typename T, int V, int SM>
__global__ __launch_bounds__(1024) void streams_kernel(sd_streams_update g, int W, float eps, int round) {
  extern __shared__ float row[];   // [W]
  __shared__ float red[32], f_mix[SM * SM], f_out[SM], f_in[SM];
  const int i = blockIdx.x, r = g.rows ? g.rows[i] : i, S = g.streams, np = W / V, nthr = blockDim.x, tid = threadIdx.x;
  float* xr = g.x + (size_t)r * S * W;
  const bool enter = g.tokens != nullptr, pair = g.b != nullptr;
  const T* erow = nullptr;
  if (enter) {
    int t = g.tokens[r];
    t = t < 0 ? 0 : (t < g.vocab ? t : g.vocab - 1);
    erow = (const T*)g.embed + (size_t)t * W;
  }
  auto load_x = [&](int c, Pack<V>* xs) {
    if (enter) {
      const Pack<V> e = ld_pack<V>(erow + c);
#pragma unroll
      for (int s = 0; s < SM; ++s) xs[s] = e;
    } else {
#pragma unroll
      for (int s = 0; s < SM; ++s)
        if (s < S) xs[s] = ld_pack<V>(xr + (size_t)s * W + c);
    }
  };
  float same = 0.f;                // what the identity experts leave of the row's own input
  if (g.sel_expert)
    for (int j = 0; j < g.n_a; ++j)
      if (g.sel_expert[(size_t)r * g.n_a + j] >= g.n_experts) same += g.sel_weight[(size_t)r * g.n_a + j];
  auto load_a = [&](int c) {
    Pack<V> y;
    if (!g.sel_expert) {
      y = ld_pack<V>(g.a + (size_t)r * g.n_a * g.lda + c);
      for (int j = 1; j < g.n_a; ++j) {
        const Pack<V> p = ld_pack<V>(g.a + ((size_t)r * g.n_a + j) * g.lda + c);
#pragma unroll
        for (int k = 0; k < V; ++k) y.v[k] += p.v[k];
      }
      return y;
    }
#pragma unroll
    for (int k = 0; k < V; ++k) y.v[k] = 0.f;
    for (int j = 0; j < g.n_a; ++j)
      if (g.sel_expert[(size_t)r * g.n_a + j] < g.n_experts) {
        const Pack<V> p = ld_pack<V>(g.a + ((size_t)r * g.n_a + j) * g.lda + c);
#pragma unroll
        for (int k = 0; k < V; ++k) y.v[k] += p.v[k];
      }
    if (same != 0.f) {
      const Pack<V> p = ld_pack<V>(g.input + (size_t)r * W + c);
#pragma unroll
      for (int k = 0; k < V; ++k) y.v[k] = fmaf(same, p.v[k], y.v[k]);
    }
    return y;
  };
  const bool mine = tid < np;
  Pack<V> x0[SM], a0, b0, wn, wa0, wb0;
  if (mine) {
    load_x(tid * V, x0);
    if (g.a) a0 = load_a(tid * V);
    if (pair) {
      b0 = ld_pack<V>(g.b + (size_t)r * g.lda + tid * V);
      wa0 = ld_pack<V>((const T*)g.w_a + tid * V);
      wb0 = ld_pack<V>((const T*)g.w_b + tid * V);
    }
    if (g.w_next) wn = ld_pack<V>((const T*)g.w_next + tid * V);
  }
  for (int c = tid; c < SM * SM; c += nthr) f_mix[c] = g.a && c / SM < S && c % SM < S ? g.mix[c / SM * S + c % SM] : 0.f;
  if (tid < SM) {
    f_out[tid] = g.a && tid < S ? g.out[tid] : 0.f;
    f_in[tid] = tid < S ? (g.in ? g.in[tid] : 1.f) : 0.f;
  }
  if (!pair) __syncthreads();      // (a pair's sums wait for all threads anyway)
  float ra = 1.f, rb = 0.f;
  if (pair) {
    float sa = 0.f, sb = 0.f;
    for (int p = tid; p < np; p += nthr) {
      const Pack<V> a = p == tid ? a0 : load_a(p * V), b = p == tid ? b0 : ld_pack<V>(g.b + (size_t)r * g.lda + p * V);
#pragma unroll
      for (int k = 0; k < V; ++k) {
        sa = fmaf(a.v[k], a.v[k], sa);
        sb = fmaf(b.v[k], b.v[k], sb);
      }
    }
    const Two s = block_sum2(sa, sb, red);
    ra = 1.f / sqrtf(s.a / (float)W + eps);
    rb = 1.f / sqrtf(s.b / (float)W + eps);
  }
  float ss = 0.f;
  for (int p = tid; p < np; p += nthr) {
    const int c = p * V;
    Pack<V> xs[SM], y;
    if (p == tid) {
#pragma unroll
      for (int s = 0; s < SM; ++s) xs[s] = x0[s];
    } else {
      load_x(c, xs);
    }
    if (g.a) {
      y = p == tid ? a0 : load_a(c);
      if (pair) {
        const Pack<V> b = p == tid ? b0 : ld_pack<V>(g.b + (size_t)r * g.lda + c);
        const Pack<V> wa = p == tid ? wa0 : ld_pack<V>((const T*)g.w_a + c);
        const Pack<V> wb = p == tid ? wb0 : ld_pack<V>((const T*)g.w_b + c);
#pragma unroll
        for (int k = 0; k < V; ++k) y.v[k] = 0.5f * (y.v[k] * ra * wa.v[k] + b.v[k] * rb * wb.v[k]);
      }
    }
    Pack<V> u, sum;
#pragma unroll
    for (int k = 0; k < V; ++k) u.v[k] = sum.v[k] = 0.f;
#pragma unroll
    for (int t = 0; t < SM; ++t)
      if (t < S) {
        Pack<V> n = xs[t];
        if (g.a) {
          const float ot = f_out[t];
#pragma unroll
          for (int k = 0; k < V; ++k) n.v[k] = 0.f;
#pragma unroll
          for (int s = 0; s < SM; ++s)
            if (s < S) {
              const float m = f_mix[s * SM + t];
#pragma unroll
              for (int k = 0; k < V; ++k) n.v[k] = fmaf(m, xs[s].v[k], n.v[k]);
            }
#pragma unroll
          for (int k = 0; k < V; ++k) n.v[k] = fmaf(ot, y.v[k], n.v[k]);
        }
        if ((g.a || enter) && !g.rows) st_pack<V>(xr + (size_t)t * W + c, n);
        const float in = f_in[t];
#pragma unroll
        for (int k = 0; k < V; ++k) {
          sum.v[k] += n.v[k];
          u.v[k] = fmaf(in, n.v[k], u.v[k]);
        }
      }
    if (g.x_copy) st_pack<V>(g.x_copy + (size_t)r * W + c, sum);
#pragma unroll
    for (int k = 0; k < V; ++k) {
      row[c + k] = u.v[k];
      ss = fmaf(u.v[k], u.v[k], ss);
    }
  }
  if (!g.w_next) return;
  const float rstd = 1.f / sqrtf(block_sum2(ss, 0.f, red).a / (float)W + eps);
  for (int p = tid; p < np; p += nthr) {
    const int c = p * V;
    const Pack<V> w = p == tid ? wn : ld_pack<V>((const T*)g.w_next + c);
    Pack<V> h;
#pragma unroll
    for (int k = 0; k < V; ++k) {
      h.v[k] = row[c + k] * rstd * (1.f + w.v[k]);
      if (round) h.v[k] = round_bf16(h.v[k]);
    }
    if (g.h) st_pack<V>(g.h + (size_t)i * W + c, h);
    if (g.h_bf16) st_pack<V>((bf16_t*)g.h_bf16 + (size_t)i * W + c, h);
  }
}

template <typename T, int V>
void launch_streams(const sd_streams_update& g, int n, int W, float eps, int round, hipStream_t st) {
  int nthr = (W / V + 63) / 64 * 64;
  if (nthr > 1024) nthr = 1024;
  const int nthr1 = W >= 1024 ? 1024 : (W + 63) / 64 * 64;
  const size_t lds = sizeof(float) * W;
  if (g.streams <= 2) streams_kernel<T, V, 2><<<n, nthr, lds, st>>>(g, W, eps, round);
  else if (g.streams <= 4) streams_kernel<T, V, 4><<<n, nthr, lds, st>>>(g, W, eps, round);
  else if (g.streams <= 8) streams_kernel<T, 1, 8><<<n, nthr1, lds, st>>>(g, W, eps, round);   // (registers)
  else streams_kernel<T, 1, 16><<<n, nthr1, lds, st>>>(g, W, eps, round);
}

// z = cap tanh(z / cap), in place
__global__ void cap_rows_kernel(float* __restrict__ x, int64_t ld, float cap, int n_cols) {
  for (int c = blockIdx.y * blockDim.x + threadIdx.x; c < n_cols; c += gridDim.y * blockDim.x) {
    float* p = x + (size_t)blockIdx.x * ld + c;
    *p = cap * tanhf(*p / cap);
  }
}

// ------------------------------------------------------------------ attention inputs with biases
struct QkvArgs {
  float* q;                // [rows, H*dk], in place
  const float* k;
  const float* v;
  int64_t ld;
  const void* q_bias;      // each [its columns] or nullptr
  const void* k_bias;
  const void* v_bias;
  const void* q_w;         // [dk]
  const void* k_w;
  void* k_cache;
  void* v_cache;
  const int32_t* row_pos;
  const int32_t* row_slot;
  const int32_t* block_tables;
  int max_blocks, page, H, G, dk, dv;
  float eps;
};
constexpr int kUnitRegs = 8;    // channels per lane at most: a head has up to 512
// One head of a row, by one wave: units 0 .. H-1 query heads (bias, norm, in place), then G key heads
// (bias, norm, appended), then G value heads (bias, appended).  NC: channels per lane (loads run unguarded, on channels clamped into the head).
template <typename T, int NC>
__device__ __forceinline__ void head_prep(const float* __restrict__ src, const T* __restrict__ bias,
                                          const T* __restrict__ w, int d, float eps, float* q_dst, T* c_dst) {
  const int lane = threadIdx.x & 63;
  float val[NC], wt[NC], bs[NC], ss = 0.f;
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = lane + 64 * k < d ? lane + 64 * k : d - 1;
    val[k] = src[c];
    bs[k] = bias ? ld_f(bias + c) : 0.f;
    wt[k] = w ? ld_f(w + c) : 1.f;
  }
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    val[k] += bs[k];
    if (lane + 64 * k < d) ss = fmaf(val[k], val[k], ss);
  }
  const float rstd = w ? 1.f / sqrtf(wave_sum(ss) / (float)d + eps) : 1.f;
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = lane + 64 * k;
    if (c < d) {
      const float o = val[k] * rstd * wt[k];
      if (q_dst) q_dst[c] = o;
      else st_f(c_dst + c, o);
    }
  }
}
template <typename T, int NC>
__device__ __forceinline__ void qkv_unit_nc(const QkvArgs& g, int r, int unit) {
  if (unit < g.H) {
    float* q = g.q + (size_t)r * g.ld + (size_t)unit * g.dk;
    head_prep<T, NC>(q, g.q_bias ? (const T*)g.q_bias + (size_t)unit * g.dk : nullptr, (const T*)g.q_w, g.dk, g.eps, q, nullptr);
    return;
  }
  const int pos = g.row_pos[r];
  const int pg = g.block_tables[(size_t)g.row_slot[r] * g.max_blocks + pos / g.page];
  unit -= g.H;
  if (unit < g.G) {
    head_prep<T, NC>(g.k + (size_t)r * g.ld + (size_t)unit * g.dk,
                     g.k_bias ? (const T*)g.k_bias + (size_t)unit * g.dk : nullptr, (const T*)g.k_w, g.dk, g.eps, nullptr,
                     (T*)g.k_cache + (((size_t)pg * g.G + unit) * g.page + pos % g.page) * g.dk);
    return;
  }
  unit -= g.G;
  head_prep<T, NC>(g.v + (size_t)r * g.ld + (size_t)unit * g.dv,
                   g.v_bias ? (const T*)g.v_bias + (size_t)unit * g.dv : nullptr, (const T*)nullptr, g.dv, g.eps, nullptr,
                   (T*)g.v_cache + (((size_t)pg * g.G + unit) * g.page + pos % g.page) * g.dv);
}
template <typename T>
__device__ __forceinline__ void qkv_unit(const QkvArgs& g, int r, int unit) {
  const int d = g.dk > g.dv ? g.dk : g.dv;
  if (d <= 64) qkv_unit_nc<T, 1>(g, r, unit);
  else if (d <= 128) qkv_unit_nc<T, 2>(g, r, unit);
  else qkv_unit_nc<T, kUnitRegs>(g, r, unit);
}
template <typename T>
__global__ __launch_bounds__(256) void qkv_prep_kernel(QkvArgs g) {
  const int unit = blockIdx.y * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  if (unit < g.H + 2 * g.G) qkv_unit<T>(g, blockIdx.x, unit);
}

// ------------------------------------------------------------------ decays from a low-rank pair
// sigmoid(b + a2 . a1)^(1/tau), through the logarithm
template <typename T>
__device__ __forceinline__ float low_rank_decay(const float* a1, const T* a2, int rank, float b, float inv_tau) {
  float z = 0.f;
  constexpr int U = 16;            // loads in flight, on indices clamped into the row
  for (int j0 = 0; j0 < rank; j0 += U) {
    float x[U], w[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int j = j0 + u < rank ? j0 + u : rank - 1;
      x[u] = a1[j];
      w[u] = ld_f(a2 + j);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (j0 + u < rank) z = fmaf(x[u], w[u], z);
  }
  return expf(log_sigmoid_f(z + b) * inv_tau);
}
// A thread per channel, kDecayRows rows per workgroup; the rows' a1 in LDS, the channel's a2 row in
// registers where it has at most RK elements (RK = 0: read as it is needed).
constexpr int kDecayRows = 8;
template <typename T, int RK>
__global__ __launch_bounds__(256) void low_rank_decay_kernel(const float* __restrict__ a1, int64_t ld,
                                                            const T* __restrict__ a2, const float* __restrict__ bias,
                                                            int rank, float inv_tau, float* __restrict__ out, int n_rows,
                                                            int n_cols) {
  extern __shared__ float as[];   // [kDecayRows][RK, or rank]
  const int r0 = blockIdx.x * kDecayRows, nr = n_rows - r0 < kDecayRows ? n_rows - r0 : kDecayRows;
  constexpr bool regs = RK > 0;
  const int lda = regs ? RK : rank;
  for (int i = threadIdx.x; i < nr * lda; i += 256) {
    const int j = i % lda;
    as[i] = j < rank ? a1[(size_t)(r0 + i / lda) * ld + j] : 0.f;
  }
  const int c = blockIdx.y * 256 + threadIdx.x, cc = c < n_cols ? c : n_cols - 1;
  const T* w = a2 + (size_t)cc * rank;
  float wr[RK > 0 ? RK : 1];
  if constexpr (RK > 0) {
    if (rank % 4 == 0) {           // (a row is then aligned to four elements, like the matrix)
#pragma unroll
      for (int j = 0; j < RK; j += 4) {
        const Pack<4> p = ld_pack<4>(w + (j < rank ? j : 0));
#pragma unroll
        for (int k = 0; k < 4; ++k) wr[j + k] = j < rank ? p.v[k] : 0.f;
      }
    } else {
#pragma unroll
      for (int j = 0; j < RK; ++j) {
        const float v = ld_f(w + (j < rank ? j : 0));
        wr[j] = j < rank ? v : 0.f;
      }
    }
  }
  const float b = bias[cc];
  __syncthreads();
  if (c >= n_cols) return;
#pragma unroll 4
  for (int i = 0; i < nr; ++i) {
    float z = 0.f;
    if constexpr (RK > 0) {
#pragma unroll
      for (int j = 0; j < RK; ++j) z = fmaf(as[i * RK + j], wr[j], z);   // (zeros behind the rank)
    } else {
      for (int j = 0; j < rank; ++j) z = fmaf(as[i * rank + j], ld_f(w + j), z);
    }
    out[(size_t)(r0 + i) * n_cols + c] = expf(log_sigmoid_f(z + b) * inv_tau);
  }
}

// ------------------------------------------------------------------ the recurrence, single tokens
// Rows that are alone in their entries (a decoding step): a workgroup per (row, head) forms the head's
// decays, moves its state on, reads it, norms and gates what was read.  A thread owns a strip of 16
// key channels of one value column (CT columns at a time).  Workgroups behind the H heads prepare the
// row's attention inputs, a wave per head.
struct StepArgs {
  sd_decay_step s;
  const int32_t* row_pos;
  const int32_t* row_slot;
  float eps;
};
constexpr int kStrip = 16;
template <typename T>
__global__ __launch_bounds__(1024) void decay_step_kernel(StepArgs a, QkvArgs g, int with_qkv, int CT, int NS) {
  extern __shared__ float lds[];
  __shared__ float red[32];
  const sd_decay_step& s = a.s;
  const int r = blockIdx.y, h = blockIdx.x, H = s.heads, dk = s.dim, dv = s.vdim, tid = threadIdx.x;
  if (h >= H) {
    const int unit = (h - H) * (blockDim.x >> 6) + __builtin_amdgcn_readfirstlane(tid >> 6);
    if (with_qkv && unit < g.H + 2 * g.G) qkv_unit<T>(g, r, unit);
    return;
  }
  float* qs = lds;                 // [NS*16]
  float* ks = qs + NS * kStrip;
  float* ds = ks + NS * kStrip;    // decays
  float* part = ds + NS * kStrip;  // [NS][CT]
  float* o = part + NS * CT;       // [dv]
  const int slot = a.row_slot[r], c = tid % CT, st = tid / CT, r0 = st * kStrip;
  const bool kept = a.row_pos[r] > 0;
  const size_t row = (size_t)r * s.ld;
  float* state = s.state + ((size_t)slot * H + h) * dk * dv;
  float S[kStrip];
  auto load = [&](int col) {       // (clamped addresses; what lies outside is zeroed or dropped)
    const int cc = col < dv ? col : dv - 1;
#pragma unroll
    for (int i = 0; i < kStrip; ++i) {
      const int rr = r0 + i < dk ? r0 + i : dk - 1;
      const float v = state[(size_t)rr * dv + cc];
      S[i] = kept && r0 + i < dk ? v : 0.f;
    }
  };
  load(c);
  for (int i = tid; i < NS * kStrip; i += blockDim.x) {
    const int cc = i < dk ? i : dk - 1, ch = h * dk + cc;
    const float d = low_rank_decay<T>(s.a1 + row, (const T*)s.a2 + (size_t)ch * s.rank, s.rank, s.a2_bias[ch], 1.f / s.tau);
    qs[i] = i < dk ? s.q[row + ch] * s.q_scale : 0.f;
    ks[i] = i < dk ? s.k[row + ch] : 0.f;
    ds[i] = d;
  }
  __syncthreads();
  for (int c0 = 0; c0 < dv; c0 += CT) {
    const int col = c0 + c;
    if (c0 > 0) load(col);
    if (st < NS) {
      const float v = s.v[row + (size_t)h * dv + (col < dv ? col : dv - 1)];
      float acc = 0.f;
#pragma unroll
      for (int i = 0; i < kStrip; ++i) {
        S[i] = fmaf(ds[r0 + i], S[i], ks[r0 + i] * v);
        acc = fmaf(S[i], qs[r0 + i], acc);
      }
      part[st * CT + c] = acc;
      if (col < dv) {
#pragma unroll
        for (int i = 0; i < kStrip; ++i)
          if (r0 + i < dk) state[(size_t)(r0 + i) * dv + col] = S[i];
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
  float ss = 0.f;
  for (int i = tid; i < dv; i += blockDim.x) ss = fmaf(o[i], o[i], ss);
  const float rstd = 1.f / sqrtf(block_sum2(ss, 0.f, red).a / (float)dv + a.eps);
  for (int i = tid; i < dv; i += blockDim.x) {
    const int ch = h * dv + i;
    const float gz = s.gate[row + ch];
    const float y = o[i] * rstd * ld_f((const T*)s.norm_w + i) * (gz * sigmoid_f(gz));
    if (s.y) s.y[(size_t)r * s.ldy + ch] = y;
    if (s.y_bf16) ((bf16_t*)s.y_bf16)[(size_t)r * s.ldy + ch] = (bf16_t)y;
  }
}

// ------------------------------------------------------------------ the recurrence, runs of tokens
// S <- diag(d_t) S + k_t v_t^T, o_t = S^T q_t over blocks of 16 tokens on the f32 matrix instruction (no
// reduced precision).  With P_t the product of the block's decays up to and including t, R_s that of
// the decays behind s, and S the state at the block's start:
//   o_t = (q_t P_t) S + sum_{s <= t} (sum_c q_t[c] k_s[c] d_{s+1}[c] .. d_t[c]) v_s
//   S  <- diag(P_last) S + (k_s R_s)^T v_s
// Every factor is a product of decays, at most one: nothing is divided, however strong the decay.  The
// inner sums of a block are formed channel by channel with running products.  A wave owns 16 value
// columns; its part of S lives in accumulators, whose layout is that of the right operand of q S as it is
// (the key channels of an MFMA step in the order the accumulators hold them).
//
// A long portion is cut into chunks of tokens that run side by side: every chunk's own sum from a zero
// state (kSums), the states at the chunks' starts (chunk_carry_kernel, chunk after chunk), then the
// tokens' results (kReads).  kWhole: a portion in one go, from and to its slot's state.
enum ChunkMode { kSums = 0, kReads = 1, kWhole = 2 };
struct ChunkArgs {
  const float* q;
  const float* k;
  const float* v;
  int64_t ld;
  const float* decay;      // [rows, H*dk]
  float q_scale;
  float* state;            // [slots, H, dk, dv]
  const int32_t* entries;
  float* out;              // [rows, H*dv]
  float* cs;               // [chunks, H, dk, dv]: own sums, then the state at the chunk's start
  float* ct;               // [chunks, H, dk]: product of the chunk's decays
  int n_entries, H, dk, dv, chunk;
};
constexpr int kBlock = 16;       // tokens of a block
constexpr int kBlockCols = 128;  // value columns per workgroup
constexpr int kTokLd = kBlock + 4;
constexpr int kChunkThreads = 512;

// The portion and the first row (inside it) of the n-th group of `per` rows over all portions.
__device__ __forceinline__ bool nth_group(const int32_t* entries, int n_entries, int per, int n, int* e, int* first) {
  int i = 0;
  for (; i < n_entries; ++i) {
    const int len = entries[4 * i + 2], groups = len / per + (len % per != 0);
    if (n < groups) break;
    n -= groups;
  }
  *e = i;
  *first = n * per;
  return i < n_entries;
}

// Up to 16 rows of up to COLS columns on their way from memory to LDS, V columns a piece.
template <int COLS, int V>
struct BlockRows {
  static constexpr int PIECES = kBlock * COLS / V, N = (PIECES + kChunkThreads - 1) / kChunkThreads;
  Pack<V> v[N];
  __device__ __forceinline__ void load(const float* src, int64_t ld, int rows, int cols) {
#pragma unroll
    for (int u = 0; u < N; ++u) {
      const int idx = threadIdx.x + kChunkThreads * u, t = idx / (COLS / V), c = idx % (COLS / V) * V;
      v[u] = ld_pack<V>(src + (size_t)(t < rows ? t : rows - 1) * ld + (c < cols ? c : cols - V));
    }
  }
  // times f; what lies outside is `pad`
  __device__ __forceinline__ void store(float* dst, int ldd, int rows, int cols, float f, float pad) {
#pragma unroll
    for (int u = 0; u < N; ++u) {
      const int idx = threadIdx.x + kChunkThreads * u, t = idx / (COLS / V), c = idx % (COLS / V) * V;
      if (PIECES % kChunkThreads != 0 && idx >= PIECES) continue;
      Pack<V> p;
#pragma unroll
      for (int e = 0; e < V; ++e) p.v[e] = t < rows && c < cols ? v[u].v[e] * f : pad;
      st_pack<V>(dst + t * ldd + c, p);
    }
  }
};

template <int DKP>
constexpr size_t decay_chunk_lds() {
  return sizeof(float) * (4 * (size_t)kBlock * (DKP + 4) + (size_t)DKP * kTokLd + DKP +
                          (size_t)kBlock * (kBlockCols + 4) + (size_t)kBlock * kTokLd);
}
template <int DKP, int V, int MODE>   // keys of up to DKP channels
__global__ __launch_bounds__(kChunkThreads, DKP <= 128 ? 4 : 2) void decay_chunk_kernel(ChunkArgs g) {
  extern __shared__ float lds[];
  constexpr int LDK = DKP + 4, LDV = kBlockCols + 4, KT = DKP / 16;
  float* qs = lds;                     // [16][LDK]
  float* ks = qs + kBlock * LDK;       // [16][LDK]
  float* ds = ks + kBlock * LDK;       // [16][LDK] decays
  float* qp = ds + kBlock * LDK;       // [16][LDK] q_t P_t
  float* kr = qp + kBlock * LDK;       // [DKP][kTokLd] k_s R_s, transposed
  float* tot = kr + DKP * kTokLd;      // [DKP] P_last
  float* vs = tot + DKP;               // [16][LDV]
  float* as = vs + kBlock * LDV;       // [16][kTokLd] the block's inner sums
  const int tid = threadIdx.x, lane = tid & 63, col = lane & 15, quad = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int dk = g.dk, dv = g.dv, H = g.H, h = blockIdx.y, c0 = blockIdx.z * kBlockCols;
  const int cols = dv - c0 < kBlockCols ? dv - c0 : kBlockCols;
  int e, first;
  if constexpr (MODE == kWhole) {
    e = blockIdx.x;
    first = 0;
  } else {
    if (!nth_group(g.entries, g.n_entries, g.chunk, blockIdx.x, &e, &first)) return;
  }
  const int slot = g.entries[4 * e], row0 = g.entries[4 * e + 1] + first, left = g.entries[4 * e + 2] - first;
  const bool kept = g.entries[4 * e + 3] > 0;
  const int nt = MODE == kWhole ? left : (left < g.chunk ? left : g.chunk);
  const size_t at = ((size_t)blockIdx.x * H + h) * dk;            // the chunk's place in ct, and (times dv) in cs
  float* slot_state = g.state + ((size_t)slot * H + h) * dk * dv + c0;
  BlockRows<DKP, V> rq, rk, rd;
  BlockRows<kBlockCols, V> rv;
  auto fetch = [&](int t0) {
    const size_t row = (size_t)(row0 + t0);
    const int n = nt - t0 < kBlock ? nt - t0 : kBlock;
    if constexpr (MODE != kSums) rq.load(g.q + row * g.ld + (size_t)h * dk, g.ld, n, dk);
    rk.load(g.k + row * g.ld + (size_t)h * dk, g.ld, n, dk);
    rd.load(g.decay + row * H * dk + (size_t)h * dk, (int64_t)H * dk, n, dk);
    rv.load(g.v + row * g.ld + (size_t)h * dv + c0, g.ld, n, cols);
  };
  fetch(0);
  const int c = 16 * wave + col;       // this wave's columns of the state; rows 16 * kt + 4 * quad + i
  const bool works = 16 * wave < cols;
  f32x4 S[KT];
#pragma unroll
  for (int kt = 0; kt < KT; ++kt) S[kt] = f32x4{0.f, 0.f, 0.f, 0.f};
  if (MODE == kReads || (MODE == kWhole && kept)) {
    const float* s0 = (MODE == kReads ? g.cs + at * dv + c0 : slot_state) + (c < cols ? c : cols - 1);
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int k = 16 * kt + 4 * quad + i;
        const float s = s0[(size_t)(k < dk ? k : dk - 1) * dv];
        S[kt][i] = k < dk && c < cols ? s : 0.f;
      }
  }
  float run = 1.f;                     // kSums: product of the chunk's decays, thread < DKP a channel
  for (int t0 = 0; t0 < nt; t0 += kBlock) {
    const int n = nt - t0 < kBlock ? nt - t0 : kBlock;
    __syncthreads();
    if constexpr (MODE != kSums) rq.store(qs, LDK, n, dk, g.q_scale, 0.f);
    rk.store(ks, LDK, n, dk, 1.f, 0.f);
    rd.store(ds, LDK, n, dk, 1.f, 1.f);
    rv.store(vs, LDV, n, cols, 1.f, 0.f);
    __syncthreads();
    if (t0 + kBlock < nt) fetch(t0 + kBlock);
    // products of decays, a thread per channel: forward, and (other threads) backward
    if (tid < DKP) {
      float d[kBlock], p = 1.f;
#pragma unroll
      for (int t = 0; t < kBlock; ++t) d[t] = ds[t * LDK + tid];
      if constexpr (MODE != kSums) {
        float q[kBlock];
#pragma unroll
        for (int t = 0; t < kBlock; ++t) q[t] = qs[t * LDK + tid];
#pragma unroll
        for (int t = 0; t < kBlock; ++t) {
          p *= d[t];
          qp[t * LDK + tid] = q[t] * p;
        }
      } else {
#pragma unroll
        for (int t = 0; t < kBlock; ++t) p *= d[t];
      }
      tot[tid] = p;
      run *= p;
    } else if (tid < 2 * DKP) {
      const int ch = tid - DKP;
      float d[kBlock], w[kBlock], p = 1.f;
#pragma unroll
      for (int t = 0; t < kBlock; ++t) {
        d[t] = ds[t * LDK + ch];
        w[t] = ks[t * LDK + ch];
      }
#pragma unroll
      for (int t = kBlock - 1; t >= 0; --t) {
        w[t] *= p;
        p *= d[t];
      }
#pragma unroll
      for (int t = 0; t < kBlock; t += 4)
        *reinterpret_cast<f32x4*>(kr + ch * kTokLd + t) = f32x4{w[t], w[t + 1], w[t + 2], w[t + 3]};
    }
    if constexpr (MODE != kSums) {
      // inner sums: this wave's tokens s = wave and wave + 8; a lane per channel; then 32 sums over 64
      // lanes, halving the number of values a lane holds at every exchange
      float a[32];
#pragma unroll
      for (int i = 0; i < 32; ++i) a[i] = 0.f;
#pragma unroll
      for (int c1 = 0; c1 < (DKP + 63) / 64; ++c1) {
        const int ch = DKP >= 64 ? lane + 64 * c1 : (lane < DKP ? lane : DKP - 1);
        float d[kBlock], q[kBlock], w[2];
#pragma unroll
        for (int t = 0; t < kBlock; ++t) {
          d[t] = ds[t * LDK + ch];
          q[t] = qs[t * LDK + ch];
        }
#pragma unroll
        for (int j = 0; j < 2; ++j) w[j] = ks[(wave + 8 * j) * LDK + ch];
        if (DKP < 64 && lane >= DKP) w[0] = w[1] = 0.f;
#pragma unroll
        for (int j = 0; j < 2; ++j)
#pragma unroll
          for (int t = 8 * j; t < kBlock; ++t) {
            const int dt = t - 8 * j;   // (against the wave's number, which is below 8)
            w[j] *= dt > 7 || dt > wave ? d[t] : 1.f;
            a[16 * j + t] = fmaf(dt > 7 || dt >= wave ? q[t] : 0.f, w[j], a[16 * j + t]);
          }
      }
#pragma unroll
      for (int b = 0; b < 5; ++b) {
        const int half = 16 >> b;
        const bool up = (lane >> b) & 1;
#pragma unroll
        for (int i = 0; i < half; ++i) {
          const float lo = a[i], hi = a[i + half];
          a[i] = (up ? hi : lo) + __shfl_xor(up ? lo : hi, 1 << b, SD_WAVE);
        }
      }
      a[0] += __shfl_xor(a[0], 32, SD_WAVE);
      const int idx = (int)(__brev((unsigned)lane) >> 27);       // the value that this lane is left with
      if (lane < 32) as[(idx & 15) * kTokLd + wave + 8 * (idx >> 4)] = a[0];
    }
    __syncthreads();
    if (!works) continue;
    f32x4 vv;
#pragma unroll
    for (int i = 0; i < 4; ++i) vv[i] = vs[(4 * quad + i) * LDV + c];
    if constexpr (MODE != kSums) {
      f32x4 o = {0.f, 0.f, 0.f, 0.f}, o2 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kt = 0; kt < KT; ++kt) {
        const f32x4 a = *reinterpret_cast<const f32x4*>(qp + col * LDK + 16 * kt + 4 * quad);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          f32x4& acc = i & 1 ? o2 : o;
          acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], S[kt][i], acc, 0, 0, 0);
        }
      }
      const f32x4 a = *reinterpret_cast<const f32x4*>(as + col * kTokLd + 4 * quad);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        f32x4& acc = i & 1 ? o2 : o;
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], vv[i], acc, 0, 0, 0);
      }
      o += o2;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = 4 * quad + i;
        if (t < n && c < cols) g.out[(size_t)(row0 + t0 + t) * H * dv + (size_t)h * dv + c0 + c] = o[i];
      }
    }
    if (MODE != kReads || t0 + kBlock < nt) {
#pragma unroll
      for (int kt = 0; kt < KT; ++kt) S[kt] *= *reinterpret_cast<const f32x4*>(tot + 16 * kt + 4 * quad);
#pragma unroll
      for (int kt = 0; kt < KT; ++kt) {
        const f32x4 a = *reinterpret_cast<const f32x4*>(kr + (16 * kt + col) * kTokLd + 4 * quad);
#pragma unroll
        for (int i = 0; i < 4; ++i) S[kt] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], vv[i], S[kt], 0, 0, 0);
      }
    }
  }
  if constexpr (MODE != kReads) {
    float* dst = MODE == kSums ? g.cs + at * dv + c0 : slot_state;
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int k = 16 * kt + 4 * quad + i;
        if (k < dk && c < cols) dst[(size_t)k * dv + c] = S[kt][i];
      }
    if (MODE == kSums && blockIdx.z == 0 && tid < dk) g.ct[at + tid] = run;
  }
}

// One element of a head's state through the chunks of its portion.
__global__ __launch_bounds__(256) void chunk_carry_kernel(ChunkArgs g) {
  const int dk = g.dk, dv = g.dv, H = g.H, h = blockIdx.y, e = blockIdx.z, x = blockIdx.x * 256 + threadIdx.x;
  if (x >= dk * dv) return;
  const int slot = g.entries[4 * e], len = g.entries[4 * e + 2];
  int first = 0;
  for (int i = 0; i < e; ++i) first += (g.entries[4 * i + 2] + g.chunk - 1) / g.chunk;
  const int nc = (len + g.chunk - 1) / g.chunk;
  float* st = g.state + ((size_t)slot * H + h) * dk * dv + x;
  float* own = g.cs + ((size_t)first * H + h) * dk * dv + x;
  const float* ct = g.ct + ((size_t)first * H + h) * dk + x / dv;
  const size_t step = (size_t)H * dk * dv, step_t = (size_t)H * dk;
  float val = g.entries[4 * e + 3] > 0 ? *st : 0.f;
  constexpr int U = 8;
  for (int i = 0; i < nc; i += U) {
    float v[U], d[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = i + u < nc ? i + u : nc - 1;
      v[u] = own[c * step];
      d[u] = ct[c * step_t];
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (i + u >= nc) break;
      own[(i + u) * step] = val;
      val = fmaf(d[u], val, v[u]);
    }
  }
  *st = val;
}

template <int DKP, int V>
hipError_t launch_decay_chunks(const ChunkArgs& c, size_t nc, hipStream_t st) {
  static std::once_flag once;
  static hipError_t err = hipSuccess;
  std::call_once(once, [] {
    const void* fns[3] = {reinterpret_cast<const void*>(decay_chunk_kernel<DKP, V, kSums>),
                          reinterpret_cast<const void*>(decay_chunk_kernel<DKP, V, kReads>),
                          reinterpret_cast<const void*>(decay_chunk_kernel<DKP, V, kWhole>)};
    for (const void* f : fns)
      if (err == hipSuccess) err = hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
  });
  if (err != hipSuccess) return err;
  constexpr size_t lds = decay_chunk_lds<DKP>();
  const unsigned z = (c.dv + kBlockCols - 1) / kBlockCols;
  if (nc == 0) {
    decay_chunk_kernel<DKP, V, kWhole><<<dim3(c.n_entries, c.H, z), kChunkThreads, lds, st>>>(c);
  } else {
    decay_chunk_kernel<DKP, V, kSums><<<dim3((unsigned)nc, c.H, z), kChunkThreads, lds, st>>>(c);
    chunk_carry_kernel<<<dim3((c.dk * c.dv + 255) / 256, c.H, c.n_entries), 256, 0, st>>>(c);
    decay_chunk_kernel<DKP, V, kReads><<<dim3((unsigned)nc, c.H, z), kChunkThreads, lds, st>>>(c);
  }
  return hipGetLastError();
}
constexpr int kChunkMin = 64, kChunkMax = 128;

int check_step(const sd_decay_step* s, const int32_t* row_pos, const int32_t* row_slot, int n_rows) {
  SD_REQUIRE(s && s->q && s->k && s->v && s->a1 && s->a2 && s->a2_bias && s->state && s->gate && s->norm_w &&
                 (s->y || s->y_bf16) && row_pos && row_slot && n_rows >= 1 && s->heads >= 1 && s->vdim >= 1 &&
                 s->rank >= 1 && s->tau > 0.f && s->ldy >= (int64_t)s->heads * s->vdim,
             SD_ERR_INVALID, "sd_decay_step_rows: bad argument");
  SD_REQUIRE(s->dim >= 1 && s->dim <= 256, SD_ERR_UNSUPPORTED, "sd_decay_step_rows: key size %d outside 1..256", s->dim);
  return SD_OK;
}
// threads and LDS of decay_step_kernel
struct StepShape { int NS, CT, nthr; size_t lds; };
StepShape step_shape(const sd_decay_step& s) {
  StepShape p;
  p.NS = (s.dim + kStrip - 1) / kStrip;
  p.CT = 1024 / p.NS;
  const int cols = (s.vdim + 15) / 16 * 16;
  if (p.CT > cols) p.CT = cols;
  if (p.CT > 128) p.CT = 128;
  p.nthr = (p.NS * p.CT + 63) / 64 * 64;
  p.lds = sizeof(float) * ((size_t)3 * p.NS * kStrip + (size_t)p.NS * p.CT + s.vdim);
  return p;
}
}  // namespace

// ====================================================================== C entry points
extern "C" int sd_streams_residual(const sd_streams_update* u, int w_f32, float eps, int n_rows, int W,
                                   int round_bf16_out, sd_stream_t stream) {
  SD_REQUIRE(u && u->x && n_rows >= 1 && W >= 1 && u->streams >= 1, SD_ERR_INVALID, "sd_streams_residual: bad argument");
  SD_REQUIRE(u->streams <= 16 && W <= 15360, SD_ERR_UNSUPPORTED, "sd_streams_residual: %d streams of width %d (at most 16 of 15360)",
             u->streams, W);
  SD_REQUIRE(!u->a || (u->mix && u->out && u->n_a >= 1 && u->lda >= W), SD_ERR_INVALID,
             "sd_streams_residual: a sublayer's result needs its mix and out factors");
  SD_REQUIRE(!u->b || (u->a && u->n_a == 1 && u->w_a && u->w_b && !u->sel_expert), SD_ERR_INVALID,
             "sd_streams_residual: a pair of results needs both and their norm weights");
  SD_REQUIRE(!u->sel_expert || (u->a && u->sel_weight && u->input), SD_ERR_INVALID,
             "sd_streams_residual: chosen experts need weights and the sublayer's input");
  SD_REQUIRE(!u->tokens || (u->embed && u->vocab >= 1 && !u->a && !u->rows), SD_ERR_INVALID,
             "sd_streams_residual: tokens need their table, and come before any sublayer");
  SD_REQUIRE(!u->w_next || u->h || u->h_bf16, SD_ERR_INVALID, "sd_streams_residual: a norm without an output");
  hipStream_t st = (hipStream_t)stream;
  const bool quad = W % 4 == 0 && u->lda % 4 == 0 && sd_aligned16(u->x) && sd_aligned16(u->a) && sd_aligned16(u->b) &&
                    sd_aligned16(u->input) && sd_aligned16(u->w_a) && sd_aligned16(u->w_b) && sd_aligned16(u->w_next) &&
                    sd_aligned16(u->x_copy) && sd_aligned16(u->h) && sd_aligned16(u->h_bf16) && sd_aligned16(u->embed);
  const int round = round_bf16_out;
  if (w_f32) {
    if (quad) launch_streams<float, 4>(*u, n_rows, W, eps, round, st);
    else launch_streams<float, 1>(*u, n_rows, W, eps, round, st);
  } else {
    if (quad) launch_streams<bf16_t, 4>(*u, n_rows, W, eps, round, st);
    else launch_streams<bf16_t, 1>(*u, n_rows, W, eps, round, st);
  }
  SD_CHECK_LAUNCH("sd_streams_residual");
  return SD_OK;
}

extern "C" int sd_cap_rows(float* x, int64_t ld, float cap, int n_rows, int n_cols, sd_stream_t stream) {
  SD_REQUIRE(x && n_rows >= 1 && n_cols >= 1 && ld >= n_cols && cap > 0.f, SD_ERR_INVALID, "sd_cap_rows: bad argument");
  int by = (n_cols + 255) / 256;
  if (by > 64) by = 64;
  cap_rows_kernel<<<dim3(n_rows, by), 256, 0, (hipStream_t)stream>>>(x, ld, cap, n_cols);
  SD_CHECK_LAUNCH("sd_cap_rows");
  return SD_OK;
}

extern "C" int sd_biased_qkv_prep(float* q, const float* k, const float* v, int64_t ld, const void* q_bias,
                                  const void* k_bias, const void* v_bias, int H, int G, int dk, int dv,
                                  const void* q_norm_w, const void* k_norm_w, int w_f32, float eps, void* k_cache,
                                  void* v_cache, const int32_t* row_pos, const int32_t* row_slot,
                                  const int32_t* block_tables, int max_blocks, int page, int n_rows,
                                  const sd_decay_step* step, sd_stream_t stream) {
  SD_REQUIRE(q && k && v && q_norm_w && k_norm_w && k_cache && v_cache && row_pos && row_slot && block_tables &&
                 max_blocks >= 1 && page >= 1 && n_rows >= 1 && H >= 1 && G >= 1,
             SD_ERR_INVALID, "sd_biased_qkv_prep: bad argument");
  SD_REQUIRE(dk >= 1 && dk <= 64 * kUnitRegs && dv >= 1 && dv <= 64 * kUnitRegs, SD_ERR_UNSUPPORTED,
             "sd_biased_qkv_prep: head sizes %d / %d outside 1..512", dk, dv);
  hipStream_t st = (hipStream_t)stream;
  QkvArgs g{q, k, v, ld, q_bias, k_bias, v_bias, q_norm_w, k_norm_w, k_cache, v_cache, row_pos, row_slot, block_tables,
            max_blocks, page, H, G, dk, dv, eps};
  const int units = H + 2 * G;
  if (step) {
    const int rc = check_step(step, row_pos, row_slot, n_rows);
    if (rc != SD_OK) return rc;
    const StepShape p = step_shape(*step);
    const int waves = p.nthr / 64;
    StepArgs a{*step, row_pos, row_slot, eps};
    const dim3 grid(step->heads + (units + waves - 1) / waves, n_rows);
    if (w_f32) decay_step_kernel<float><<<grid, p.nthr, p.lds, st>>>(a, g, 1, p.CT, p.NS);
    else decay_step_kernel<bf16_t><<<grid, p.nthr, p.lds, st>>>(a, g, 1, p.CT, p.NS);
  } else {
    const dim3 grid(n_rows, (units + 3) / 4);
    if (w_f32) qkv_prep_kernel<float><<<grid, 256, 0, st>>>(g);
    else qkv_prep_kernel<bf16_t><<<grid, 256, 0, st>>>(g);
  }
  SD_CHECK_LAUNCH("sd_biased_qkv_prep");
  return SD_OK;
}

extern "C" int sd_decay_step_rows(const sd_decay_step* step, int w_f32, float eps, const int32_t* row_pos,
                                  const int32_t* row_slot, int n_rows, sd_stream_t stream) {
  const int rc = check_step(step, row_pos, row_slot, n_rows);
  if (rc != SD_OK) return rc;
  const StepShape p = step_shape(*step);
  StepArgs a{*step, row_pos, row_slot, eps};
  QkvArgs none{};
  hipStream_t st = (hipStream_t)stream;
  const dim3 grid(step->heads, n_rows);
  if (w_f32) decay_step_kernel<float><<<grid, p.nthr, p.lds, st>>>(a, none, 0, p.CT, p.NS);
  else decay_step_kernel<bf16_t><<<grid, p.nthr, p.lds, st>>>(a, none, 0, p.CT, p.NS);
  SD_CHECK_LAUNCH("sd_decay_step_rows");
  return SD_OK;
}

extern "C" int sd_low_rank_decay(const float* a1, int64_t ld, const void* a2, const float* a2_bias, int w_f32, int rank,
                                 float tau, float* out, int n_rows, int n_cols, sd_stream_t stream) {
  SD_REQUIRE(a1 && a2 && a2_bias && out && n_rows >= 1 && n_cols >= 1 && rank >= 1 && ld >= rank && tau > 0.f,
             SD_ERR_INVALID, "sd_low_rank_decay: bad argument");
  SD_REQUIRE(rank <= 1536, SD_ERR_UNSUPPORTED, "sd_low_rank_decay: rank %d above 1536", rank);
  SD_REQUIRE(sd_aligned16(a2), SD_ERR_INVALID, "sd_low_rank_decay: a2 unaligned");
  const dim3 grid((n_rows + kDecayRows - 1) / kDecayRows, (n_cols + 255) / 256);
  const size_t lds = sizeof(float) * kDecayRows * (rank <= 16 ? 16 : (rank <= 64 ? 64 : rank));
  hipStream_t st = (hipStream_t)stream;
#define SD_GO(T)                                                                                                        \
  do {                                                                                                                  \
    if (rank <= 16) low_rank_decay_kernel<T, 16><<<grid, 256, lds, st>>>(a1, ld, (const T*)a2, a2_bias, rank, 1.f / tau, out, n_rows, n_cols); \
    else if (rank <= 64) low_rank_decay_kernel<T, 64><<<grid, 256, lds, st>>>(a1, ld, (const T*)a2, a2_bias, rank, 1.f / tau, out, n_rows, n_cols); \
    else low_rank_decay_kernel<T, 0><<<grid, 256, lds, st>>>(a1, ld, (const T*)a2, a2_bias, rank, 1.f / tau, out, n_rows, n_cols); \
  } while (0)
  if (w_f32) SD_GO(float);
  else SD_GO(bf16_t);
#undef SD_GO
  SD_CHECK_LAUNCH("sd_low_rank_decay");
  return SD_OK;
}

extern "C" size_t sd_decay_chunks_scratch_bytes(int n_rows, int n_entries, int H, int dk, int dv) {
  // (rows that fill no more than a chunk beyond one per portion run in one go)
  if (n_rows < 1 || n_entries < 1 || n_rows - n_entries < kChunkMin || H < 1 || dk < 1 || dv < 1) return 0;
  return sizeof(float) * ((size_t)n_rows / kChunkMin + n_entries) * H * ((size_t)dk * dv + dk);
}

extern "C" int sd_decay_chunks(const float* q, const float* k, const float* v, int64_t ld, const float* decay,
                               float q_scale, float* state, const int32_t* entries, int n_entries, int n_rows, float* out,
                               int H, int dk, int dv, void* scratch, size_t scratch_bytes, sd_stream_t stream) {
  SD_REQUIRE(q && k && v && decay && state && entries && out && n_entries >= 1 && n_rows >= n_entries && H >= 1 && dv >= 1,
             SD_ERR_INVALID, "sd_decay_chunks: bad argument");
  SD_REQUIRE(dk >= 1 && dk <= 256, SD_ERR_UNSUPPORTED, "sd_decay_chunks: key size %d outside 1..256", dk);
  const size_t need = sd_decay_chunks_scratch_bytes(n_rows, n_entries, H, dk, dv);
  const bool cut = need > 0 && scratch && scratch_bytes >= need && sd_aligned16(scratch);
  ChunkArgs c{q, k, v, ld, decay, q_scale, state, entries, out, nullptr, nullptr, n_entries, H, dk, dv, kChunkMin};
  size_t nc = 0;
  if (cut) {
    // (longer chunks, and so less carried state, where they still fill the chip)
    const long long wgs = (long long)(n_rows / kChunkMax) * H * ((dv + kBlockCols - 1) / kBlockCols);
    c.chunk = wgs >= 256 ? kChunkMax : kChunkMin;
    nc = (size_t)n_rows / c.chunk + n_entries;
    c.cs = (float*)scratch;
    c.ct = c.cs + nc * H * dk * dv;
  }
  const bool quad = ld % 4 == 0 && dk % 4 == 0 && dv % 4 == 0 && sd_aligned16(q) && sd_aligned16(k) && sd_aligned16(v) &&
                    sd_aligned16(decay);
  hipStream_t st = (hipStream_t)stream;
  hipError_t err;
#define SD_GO(D) err = quad ? launch_decay_chunks<D, 4>(c, nc, st) : launch_decay_chunks<D, 1>(c, nc, st)
  if (dk <= 32) SD_GO(32);
  else if (dk <= 64) SD_GO(64);
  else if (dk <= 128) SD_GO(128);
  else SD_GO(256);
#undef SD_GO
  SD_REQUIRE(err == hipSuccess, SD_ERR_HIP, "sd_decay_chunks: launch failed: %s", hipGetErrorString(err));
  return SD_OK;
}
