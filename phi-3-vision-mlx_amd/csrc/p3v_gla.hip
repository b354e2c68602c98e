// Gated linear attention: a recurrence with a [dim, vdim] state per head and a decay per key channel,
//
//   S_t = diag(a_t) S_{t-1} + k_t v_t^T,   o_t = S_t^T q_t,   a = sigmoid(W_a2 a1 + b)^(1 / tau),
//
// then an RMS norm of o over vdim and a SiLU gate.  Everything that enters the recurrence is fp32 (the products run on the fp32 matrix
// cores), whatever the activations' type; the states are fp32.
//
// One new token: a workgroup per (head, sequence) reads the state out of the ring's slot past % R and writes the next slot.
// A prompt: chunks of 64 tokens in three launches --
//   k_gla_chunk   per chunk: the decays c_t (running sums of log2 a), what the chunk's tokens leave in the state,
//                 sum_s (k_s 2^(c_end - c_s)) v_s^T, and the whole chunk's decay 2^c_end
//   k_gla_scan    per state element: the states at the chunks' starts, in order
//   k_gla_out     per chunk: (q_t 2^c_t) S_start + sum_{s <= t} (q_t . k_s 2^(c_t - c_s)) v_s, norm, gate
// No decay is too strong for it: an exponential is taken of c_t - c_s with s <= t only, never positive.  Across the 16-token blocks of a
// chunk both factors refer to the later block's start; inside a block the keys' factor would be positive, so a block over which some
// channel decays by more than 2^GLA_SAFE takes its exponentials pair by pair.
#include "p3v_layered.h"

#define GLA_C 64                     // tokens of a chunk
#define GLA_LOG2E 1.4426950408889634f

struct GlaP {
  const void* y; const bf16_t* a2; const bf16_t* a2b; const bf16_t* norm; float* s; void* out; float* ws;
  const int32_t* pad_len; const int32_t* d_past;
  float eps, inv_tau, q_scale;
  int B, L, H, dim, vdim, rank, ld, past, R, keep, n_tok, store;
};

// workgroup barrier for LDS data only: global loads stay in flight across it
__device__ __forceinline__ void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}
// log2 of the decay, from z = W_a2 a1 + b: log sigmoid(z) = min(z, 0) - log(1 + x) with x = e^-|z|, the rounding of 1 + x given back
__device__ __forceinline__ float log2_decay(float z, float inv_tau) {
  const float x = __builtin_amdgcn_exp2f(-fabsf(z) * GLA_LOG2E), u = 1.f + x;
  const float l = __builtin_amdgcn_logf(u) + (x - (u - 1.f)) * GLA_LOG2E * __builtin_amdgcn_rcpf(u);
  return (fminf(z, 0.f) * GLA_LOG2E - l) * inv_tau;
}
// 2^x - 1 for -1 < x <= 0, 2^x below: what a step multiplies a state with, next to the state itself or next to nothing.  (A slow decay is
// 1 - tiny: rounded to fp32 before it meets the state, it would be off by up to 2^-25 in every step, the same way each time.)
__device__ __forceinline__ float decay_less_one(float x) {
  if (x <= -1.f) return __builtin_amdgcn_exp2f(x);
  const float t = x * 0.6931471805599453f;
  const float series = t * fmaf(t, fmaf(t, fmaf(t, fmaf(t, 1.f / 120.f, 1.f / 24.f), 1.f / 6.f), 0.5f), 1.f);
  return t > -0.03f ? series : __builtin_amdgcn_exp2f(x) - 1.f;
}
__device__ __forceinline__ float silu32(float g) { return g / (1.f + expf(-g)); }

// ================================================================ token by token: one new token, and any sizes
// V consecutive value columns per thread, the threads' groups share the key channels; the state of token l is read from where token
// l - 1 left it (tokens that do not stay: scratch).
#define GLA_PRE 8
template <typename T, int V>
__global__ void __launch_bounds__(512) k_gla_steps(GlaP p) {
  extern __shared__ float sm[];
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x, dim = p.dim, vdim = p.vdim;
  const int nc = (vdim + V - 1) / V, ng = max(1, 512 / nc);
  float *q = sm, *k = q + dim, *al = k + dim, *rest = al + dim, *v = rest + dim, *po = v + vdim;      // po [ng][vdim]
  __shared__ float red[8];
  const int past = p.d_past ? *p.d_past : p.past, first = p.pad_len ? p.pad_len[b] : 0;
  const size_t head = (size_t)dim * vdim, at = (size_t)b * p.R * p.H + h;
  float* ring = p.s;
  auto slot = [&](int t) { return ring + (at + (size_t)(t % p.R) * p.H) * head; };
  float* stay = slot(past + p.keep);
  float* scratch = p.ws ? p.ws + ((size_t)b * p.H + h) * head : nullptr;
  const float* src = slot(past);
  const int dg = tid / nc, c = (tid - dg * nc) * V;
  const bool mine = dg < ng;
  for (int l = 0; l < p.L; ++l) {
    const int pos = past + l;
    float* dst = l < p.keep ? stay : scratch;
    const bool live = pos >= first, fresh = pos <= first;        // (a sequence's first token finds no state)
    float st[GLA_PRE][V];
    if (mine) {
#pragma unroll
      for (int i = 0; i < GLA_PRE; ++i) {
        const int d = dg + i * ng;
#pragma unroll
        for (int j = 0; j < V; ++j) st[i][j] = 0.f;
        if (d < dim && !fresh) {
          if constexpr (V == 4) { const float4 x = *(const float4*)(src + (size_t)d * vdim + c); st[i][0] = x.x, st[i][1] = x.y, st[i][2] = x.z, st[i][3] = x.w; }
          else st[i][0] = src[(size_t)d * vdim + c];
        }
      }
    }
    const T* row = (const T*)p.y + ((size_t)b * p.L + l) * p.ld;
    const T* a1 = row + 2 * p.H * (dim + vdim);
    for (int d = tid; d < dim; d += 512) {
      q[d] = load_act(row + h * dim + d) * p.q_scale;
      k[d] = load_act(row + (p.H + h) * dim + d);
      float z = bf16_to_f32(p.a2b[h * dim + d]);
      const bf16_t* w = p.a2 + (size_t)(h * dim + d) * p.rank;
      int r = 0;
      for (; r + 16 <= p.rank; r += 16) {                        // (sixteen at a time: all loads in flight)
        float wr[16], ar[16];
#pragma unroll
        for (int j = 0; j < 16; ++j) wr[j] = bf16_to_f32(w[r + j]), ar[j] = load_act(a1 + r + j);
#pragma unroll
        for (int j = 0; j < 16; ++j) z = fmaf(wr[j], ar[j], z);
      }
      for (; r < p.rank; ++r) z = fmaf(bf16_to_f32(w[r]), load_act(a1 + r), z);
      const float x = log2_decay(z, p.inv_tau);
      al[d] = decay_less_one(x), rest[d] = x > -1.f ? 1.f : 0.f;
    }
    for (int i = tid; i < vdim; i += 512) v[i] = load_act(row + 2 * p.H * dim + h * vdim + i);
    __syncthreads();
    if (mine) {
      float o[V], vv[V];
#pragma unroll
      for (int j = 0; j < V; ++j) o[j] = 0.f, vv[j] = v[c + j];
      auto update = [&](int d, float (&x)[V]) {
        const float a = al[d], kd = k[d], qd = q[d], one = rest[d];
#pragma unroll
        for (int j = 0; j < V; ++j) {
          x[j] = live ? fmaf(a, x[j], fmaf(one, x[j], kd * vv[j])) : 0.f;
          o[j] = fmaf(qd, x[j], o[j]);
        }
        if (dst) {
          if constexpr (V == 4) *(float4*)(dst + (size_t)d * vdim + c) = make_float4(x[0], x[1], x[2], x[3]);
          else dst[(size_t)d * vdim + c] = x[0];
        }
      };
#pragma unroll
      for (int i = 0; i < GLA_PRE; ++i)
        if (dg + i * ng < dim) update(dg + i * ng, st[i]);
      for (int d = dg + GLA_PRE * ng; d < dim; d += ng) {
        float x[V];
#pragma unroll
        for (int j = 0; j < V; ++j) x[j] = fresh ? 0.f : src[(size_t)d * vdim + c + j];
        update(d, x);
      }
#pragma unroll
      for (int j = 0; j < V; ++j) po[dg * vdim + c + j] = o[j];
    }
    __syncthreads();
    float ss = 0.f;
    for (int i = tid; i < vdim; i += 512) {
      float o = 0.f;
      for (int g = 0; g < ng; ++g) o += po[g * vdim + i];
      v[i] = o;
      ss += o * o;
    }
    const float r = 1.f / sqrtf(block_sum(ss, red) / (float)vdim + p.eps);
    const T* gate = row + 2 * p.H * dim + (p.H + h) * vdim;
    T* out = (T*)p.out + ((size_t)b * p.L + l) * p.H * vdim + h * vdim;
    for (int i = tid; i < vdim; i += 512) store_act(out + i, v[i] * r * bf16_to_f32(p.norm[i]) * silu32(load_act(gate + i)));
    src = dst;
    __syncthreads();
  }
}

// ================================================================ prompts: chunks
// the live tokens [lo, hi) of a chunk
__device__ __forceinline__ void gla_span(const GlaP& p, int b, int l0, int& lo, int& hi) {
  const int past = p.d_past ? *p.d_past : p.past, first = p.pad_len ? p.pad_len[b] : 0;
  lo = min(max(first - past - l0, 0), GLA_C);
  hi = max(min(p.n_tok - l0, GLA_C), lo);
}
// LDS row strides (elements): token rows of channels (16 rows of 4 floats in distinct banks), channel rows of tokens
__host__ __device__ __forceinline__ int gla_dim16(int n) { return (n + 15) / 16 * 16; }
__host__ __device__ __forceinline__ int gla_stride(int n) { return gla_dim16(n) + 4; }
#define GLA_TS (GLA_C + 4)
__host__ __device__ __forceinline__ int gla_key_rows(int dim) { return max(gla_dim16(dim), 32); }     // (also the scratch of gla_decays)
// workspace: states [chunk, B, H, dim, vdim], decays of whole chunks [chunk, B, H, dim], running sums [B L, H, dim]
__host__ __device__ __forceinline__ size_t gla_decay_at(const GlaP& p, int nc) { return (size_t)nc * p.B * p.H * p.dim * p.vdim; }
__host__ __device__ __forceinline__ size_t gla_sums_at(const GlaP& p, int nc) { return gla_decay_at(p, nc) + (size_t)nc * p.B * p.H * p.dim; }

// c[t][d] (row stride S) = sum of log2 a over the chunk's tokens up to t, 256 threads.  a1: LDS scratch of 64 x 20 floats.  Tokens that
// are none (padding, behind the end) decay nothing.
template <typename T>
__device__ __forceinline__ void gla_decays(const GlaP& p, int b, int h, int l0, int lo, int hi, float* c, int S, float* a1) {
  const int tid = threadIdx.x, dim = p.dim;
  int G = 1;
  while (G < 16 && 2 * G * dim <= 256) G *= 2;
  const int per = GLA_C / G, d = tid % dim, g = tid / dim;
  const bool mine = g < G;
  const T* base = (const T*)p.y + ((size_t)b * p.L + l0) * p.ld + 2 * p.H * (dim + p.vdim);
  for (int r0 = 0; r0 < p.rank; r0 += 16) {
    const int nr = min(16, p.rank - r0);
    if (r0) lds_barrier();
#pragma unroll
    for (int i = 0; i < GLA_C * 16 / 256; ++i) {
      const int t = (tid >> 4) + i * 16, r = tid & 15;
      a1[t * 20 + r] = t >= lo && t < hi && r < nr ? load_act(base + (size_t)t * p.ld + r0 + r) : 0.f;
    }
    float w[16];
    if (mine) {
#pragma unroll
      for (int r = 0; r < 16; ++r) w[r] = r < nr ? bf16_to_f32(p.a2[(size_t)(h * dim + d) * p.rank + r0 + r]) : 0.f;
    }
    lds_barrier();
    if (mine) {
      const float bias = bf16_to_f32(p.a2b[h * dim + d]);
      const bool last = r0 + 16 >= p.rank;
      float run = 0.f;
      for (int t = g * per; t < (g + 1) * per; ++t) {
        float z = r0 == 0 ? bias : c[t * S + d];
#pragma unroll
        for (int r = 0; r < 16; r += 4) {
          const float4 x = *(const float4*)(a1 + t * 20 + r);
          z = fmaf(w[r], x.x, z), z = fmaf(w[r + 1], x.y, z), z = fmaf(w[r + 2], x.z, z), z = fmaf(w[r + 3], x.w, z);
        }
        if (last) {
          run += t >= lo && t < hi ? log2_decay(z, p.inv_tau) : 0.f;
          z = run;
        }
        c[t * S + d] = z;
      }
    }
  }
  lds_barrier();
  float off = 0.f;
  if (mine)
    for (int i = 0; i < g; ++i) off += c[((i + 1) * per - 1) * S + d];
  lds_barrier();
  if (mine && g > 0)
    for (int t = g * per; t < (g + 1) * per; ++t) c[t * S + d] += off;
  lds_barrier();
}

// Rows of 64 tokens, NC x 64 channels at most, through registers (requested early, written to LDS late).  A wave takes 32 tokens x 16 channels,
// 8 channels a lane: transposed LDS writes then fall into distinct banks.  Dead tokens and channels behind n are zero.
template <typename T, int NC> struct GlaRows {
  static constexpr int W = (int)sizeof(T) / 2;                           // 16-byte pieces of 8 values
  u32x4_t x[NC][2][W];
  __device__ __forceinline__ void load(const T* src, int ld, int n, int lo, int hi, int tid) {
    const int t8 = tid & 31, c8 = (tid >> 5) * 8;
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const int t = t8 + 32 * i, c0 = c * 64 + c8;
        const bool live = t >= lo && t < hi && c0 < n;
#pragma unroll
        for (int j = 0; j < W; ++j) {
          x[c][i][j] = (u32x4_t){0u, 0u, 0u, 0u};
          if (live) x[c][i][j] = *(const u32x4_t*)(src + (size_t)t * ld + c0 + j * (8 / W));
        }
      }
  }
  __device__ __forceinline__ float get(int c, int i, int j) const {
    if constexpr (W == 1) return j & 1 ? bf16hi(x[c][i][0][j >> 1]) : bf16lo(x[c][i][0][j >> 1]);
    else return __uint_as_float(x[c][i][j >> 2][j & 3]);
  }
  __device__ __forceinline__ T raw(int c, int i, int j) const {
    if constexpr (W == 1) return (T)(x[c][i][0][j >> 1] >> (16 * (j & 1)));
    else return __uint_as_float(x[c][i][j >> 2][j & 3]);
  }
  // channel rows of tokens, row stride GLA_TS
  __device__ __forceinline__ void put_transposed(T* dst, int n, int tid) const {
    const int t8 = tid & 31, c8 = (tid >> 5) * 8;
#pragma unroll
    for (int c = 0; c < NC; ++c)
      if (c * 64 + c8 < gla_dim16(n))
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
          for (int j = 0; j < 8; ++j) dst[(c * 64 + c8 + j) * GLA_TS + t8 + 32 * i] = raw(c, i, j);
  }
};

// The fp32 MFMA takes one k per lane group; four of them in a row are given k = 4 group + 0 .. 3 of a run of 16, so that an operand's four
// values are one LDS read.
// NK, NV: 64-channel groups of a key, of a value
template <typename T, int NK, int NV>
__global__ void __launch_bounds__(256) k_gla_chunk(GlaP p) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  const int ch = blockIdx.x, h = blockIdx.y, b = blockIdx.z, tid = threadIdx.x, lane = tid & 63, lc = lane & 15, lg = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int dim = p.dim, vdim = p.vdim, DS = gla_stride(dim), l0 = ch * GLA_C;
  float *cum = (float*)smem, *kd = cum + GLA_C * DS;                     // [64][DS], [dim16][TS]
  T* vt = (T*)(kd + gla_key_rows(dim) * GLA_TS);                           // [vdim16][TS]
  int lo, hi;
  gla_span(p, b, l0, lo, hi);
  const T* base = (const T*)p.y + ((size_t)b * p.L + l0) * p.ld;
  GlaRows<T, NK> kx;
  GlaRows<T, NV> vx;
  vx.load(base + 2 * p.H * dim + h * vdim, p.ld, vdim, lo, hi, tid);
  kx.load(base + (p.H + h) * dim, p.ld, dim, lo, hi, tid);
  gla_decays<T>(p, b, h, l0, lo, hi, cum, DS, kd);
  vx.put_transposed(vt, vdim, tid);
  const size_t row = (size_t)ch * p.B * p.H + (size_t)b * p.H + h;
  float* decay = p.ws + gla_decay_at(p, gridDim.x) + row * dim;
  float* sums = p.ws + gla_sums_at(p, gridDim.x) + ((size_t)b * p.L + l0) * p.H * dim + h * dim;
  const int t8 = tid & 31, c8 = (tid >> 5) * 8;
#pragma unroll
  for (int n = 0; n < NK; ++n) {
    const int c0 = n * 64 + c8;
    if (c0 >= gla_dim16(dim)) continue;
    float end[8] = {};
    if (c0 < dim) load_acts<8>(cum + (GLA_C - 1) * DS + c0, end);
    if (t8 == 0 && c0 < dim)
#pragma unroll
      for (int j = 0; j < 8; ++j) decay[c0 + j] = __builtin_amdgcn_exp2f(end[j]);
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int t = t8 + 32 * i;
      float c[8] = {};
      if (c0 < dim) load_acts<8>(cum + t * DS + c0, c);
      if (l0 + t < p.L && c0 < dim) store_acts<8>(sums + (size_t)t * p.H * dim + c0, c);
#pragma unroll
      for (int j = 0; j < 8; ++j) kd[(c0 + j) * GLA_TS + t] = kx.get(n, i, j) * __builtin_amdgcn_exp2f(fminf(end[j] - c[j], 0.f));
    }
  }
  __syncthreads();
  // A operand: row = key channel; B operand: column = value channel; a wave takes consecutive tiles, the keys of a row of them stay
  const int VT = (vdim + 15) / 16, tiles = (dim + 15) / 16 * VT, per = (tiles + 3) / 4;
  float* dst = p.ws + row * dim * vdim;
  float ka[4][4];
  int have = -1;
  for (int u = wave * per; u < min((wave + 1) * per, tiles); ++u) {
    const int dt = u / VT, v0 = (u - dt * VT) * 16;
    if (dt != have) {
#pragma unroll
      for (int q = 0; q < 4; ++q) load4(kd + (dt * 16 + lc) * GLA_TS + q * 16 + lg * 4, ka[q]);
      have = dt;
    }
    f32x4_t acc = {0.f, 0.f, 0.f, 0.f}, acc2 = {0.f, 0.f, 0.f, 0.f};     // (two chains: the products do not wait for each other)
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      float vb[4];
      load4(vt + (v0 + lc) * GLA_TS + q * 16 + lg * 4, vb);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        if (q & 1) acc2 = __builtin_amdgcn_mfma_f32_16x16x4f32(ka[q][i], vb[i], acc2, 0, 0, 0);
        else acc = __builtin_amdgcn_mfma_f32_16x16x4f32(ka[q][i], vb[i], acc, 0, 0, 0);
      }
    }
    if (v0 + lc < vdim)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (dt * 16 + lg * 4 + r < dim) dst[(size_t)(dt * 16 + lg * 4 + r) * vdim + v0 + lc] = acc[r] + acc2[r];
  }
}

// the chunks' contributions -> the states at their starts, in place; the state behind the last one goes into the ring
__global__ void __launch_bounds__(256) k_gla_scan(GlaP p, int nc) {
  constexpr int U = 8;
  const int per = p.dim * p.vdim / 4, i = blockIdx.x * 256 + threadIdx.x, bh = blockIdx.y, b = bh / p.H, h = bh - b * p.H;
  if (i >= per) return;
  const int past = p.d_past ? *p.d_past : p.past, first = p.pad_len ? p.pad_len[b] : 0;
  const size_t head = (size_t)p.dim * p.vdim, step = (size_t)p.B * p.H * head, dstep = (size_t)p.B * p.H * p.dim;
  float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
  if (past > first) s = *(const float4*)(p.s + (((size_t)b * p.R + past % p.R) * p.H + h) * head + 4 * i);
  float* a = p.ws + (size_t)bh * head + 4 * i;
  const float* dc = p.ws + gla_decay_at(p, nc) + (size_t)bh * p.dim + 4 * i / p.vdim;
  for (int c0 = 0; c0 < nc; c0 += U) {
    float4 x[U];
    float e[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = min(c0 + u, nc - 1);
      x[u] = *(const float4*)(a + c * step);
      e[u] = dc[c * dstep];
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (c0 + u < nc) {
        *(float4*)(a + (c0 + u) * step) = s;
        s = make_float4(fmaf(e[u], s.x, x[u].x), fmaf(e[u], s.y, x[u].y), fmaf(e[u], s.z, x[u].z), fmaf(e[u], s.w, x[u].w));
      }
  }
  if (p.store) *(float4*)(p.s + (((size_t)b * p.R + (past + p.n_tok) % p.R) * p.H + h) * head + 4 * i) = s;
}

// Wave w owns the chunk's tokens 16 w .. 16 w + 15, one per lane column; everything is transposed: pairs [s, t] and outputs [v, t], so that a
// lane's pairs are the operand of the product with the values as they lie.  VT: 16-channel tiles of a value.
#define GLA_SAFE 60.f
template <typename T, int VT>
__global__ void __launch_bounds__(256, VT <= 8 ? 3 : 2) k_gla_out(GlaP p) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  const int ch = blockIdx.x, h = blockIdx.y, b = blockIdx.z, tid = threadIdx.x, lane = tid & 63, lc = lane & 15, lg = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int dim = p.dim, vdim = p.vdim, DS = gla_stride(dim), l0 = ch * GLA_C, t0 = wave * 16;
  float* cum = (float*)smem;                                             // [64][DS]
  T *k = (T*)(cum + GLA_C * DS), *vt = k + GLA_C * DS;                   // [64][DS], [vdim16][TS]
  int lo, hi;
  gla_span(p, b, l0, lo, hi);
  const T* base = (const T*)p.y + ((size_t)b * p.L + l0) * p.ld;
  const float* sums = p.ws + gla_sums_at(p, gridDim.x) + ((size_t)b * p.L + l0) * p.H * dim + h * dim;
  GlaRows<T, (VT + 3) / 4> vx;
  vx.load(base + 2 * p.H * dim + h * vdim, p.ld, vdim, lo, hi, tid);
  const int n4 = gla_dim16(dim) / 4, t4 = tid >> 4;
  for (int c = tid & 15; c < n4; c += 16)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = t4 + 16 * i;
      float x[4] = {0.f, 0.f, 0.f, 0.f}, y[4] = {0.f, 0.f, 0.f, 0.f};
      if (l0 + t < p.L && 4 * c < dim) load4(sums + (size_t)t * p.H * dim + 4 * c, x);
      if (t >= lo && t < hi && 4 * c < dim) load4(base + (size_t)t * p.ld + (p.H + h) * dim + 4 * c, y);
      store4(cum + t * DS + 4 * c, x), store4(k + t * DS + 4 * c, y);
    }
  vx.put_transposed(vt, vdim, tid);
  const int l = min(l0 + t0 + lc, p.L - 1);                              // this lane's token
  const T* q = (const T*)p.y + ((size_t)b * p.L + l) * p.ld + h * dim;
  const float* S = p.ws + ((size_t)ch * p.B * p.H + (size_t)b * p.H + h) * dim * vdim;
  struct { float q[4], s[VT][4]; } x;                                    // query and starting state of 16 key channels
  auto request = [&](int d0) {
    const int d = d0 + 4 * lg;
    x.q[0] = x.q[1] = x.q[2] = x.q[3] = 0.f;
    if (d < dim) load4(q + d, x.q);
#pragma unroll
    for (int j = 0; j < VT; ++j)
#pragma unroll
      for (int i = 0; i < 4; ++i) x.s[j][i] = S[(size_t)min(d + i, dim - 1) * vdim + min(j * 16 + lc, vdim - 1)];
  };
  request(0);
  lds_barrier();
  const float* ref = cum + max(t0 - 1, 0) * DS;                          // decays before this block (wave 0: none)
  bool strong = false;                                                   // does some channel decay too much over the block?
  const int tl = min(t0 + 15, p.L - 1 - l0);                             // its last row in memory
  if (tl >= t0)
    for (int d = lane; d < dim; d += 64) strong |= (wave ? ref[d] : 0.f) - cum[tl * DS + d] > GLA_SAFE;
  strong = __builtin_amdgcn_ballot_w64(strong) != 0;

  f32x4_t sc[4], o[VT];
#pragma unroll
  for (int j = 0; j < 4; ++j) sc[j] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int j = 0; j < VT; ++j) o[j] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
  for (int d0 = 0; d0 < dim; d0 += 16) {
    if (d0) request(d0);                                                 // (not a step ahead: the registers are worth more as occupancy)
    const int d = d0 + 4 * lg;
    float qv[4], ct[4], rf[4] = {0.f, 0.f, 0.f, 0.f}, qd[4];
    load4(cum + (t0 + lc) * DS + d, ct);
    if (wave) load4(ref + d, rf);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      qv[i] = x.q[i] * p.q_scale * __builtin_amdgcn_exp2f(fminf(ct[i] - rf[i], 0.f));
      qd[i] = qv[i] * __builtin_amdgcn_exp2f(rf[i]);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j < wave || (j == wave && !strong)) {
        float kb[4], cs[4];
        load4(k + (j * 16 + lc) * DS + d, kb), load4(cum + (j * 16 + lc) * DS + d, cs);
#pragma unroll
        for (int i = 0; i < 4; ++i) kb[i] *= __builtin_amdgcn_exp2f(rf[i] - cs[i]);
#pragma unroll
        for (int i = 0; i < 4; ++i) sc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(kb[i], qv[i], sc[j], 0, 0, 0);
      }
#pragma unroll
    for (int j = 0; j < VT; ++j)
#pragma unroll
      for (int i = 0; i < 4; ++i) o[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.s[j][i], qd[i], o[j], 0, 0, 0);
  }
#pragma unroll
  for (int j = 0; j < 4; ++j)
    if (j == wave) {                                                     // the block's own pairs: s <= t
      if (strong) {
        for (int d = 0; d < dim; ++d) {
          const float qs = load_act(q + d) * p.q_scale, ct = cum[(t0 + lc) * DS + d];
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int s = (t0 + lg * 4 + r) * DS + d;
            sc[j][r] = fmaf(qs * load_act(k + s), __builtin_amdgcn_exp2f(fminf(ct - cum[s], 0.f)), sc[j][r]);
          }
        }
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) sc[j][r] = lg * 4 + r <= lc ? sc[j][r] : 0.f;
    }
#pragma unroll
  for (int j = 0; j < 4; ++j)
    if (j <= wave) {
#pragma unroll
      for (int v = 0; v < VT; ++v) {
        float va[4];
        load4(vt + min(v * 16 + lc, gla_dim16(vdim) - 1) * GLA_TS + j * 16 + lg * 4, va);
#pragma unroll
        for (int i = 0; i < 4; ++i) o[v] = __builtin_amdgcn_mfma_f32_16x16x4f32(va[i], sc[j][i], o[v], 0, 0, 0);
      }
    }
  // ---- norm over the value channels, gate
  float ss = 0.f;
#pragma unroll
  for (int v = 0; v < VT; ++v)
#pragma unroll
    for (int r = 0; r < 4; ++r) ss += v * 16 + lg * 4 + r < vdim ? o[v][r] * o[v][r] : 0.f;
  const float rs = 1.f / sqrtf(rows_sum(ss) / (float)vdim + p.eps);
  if (l0 + t0 + lc >= p.L) return;
  const T* gate = base + (size_t)(t0 + lc) * p.ld + 2 * p.H * dim + (p.H + h) * vdim;
  T* out = (T*)p.out + ((size_t)b * p.L + l) * p.H * vdim + (size_t)h * vdim;
#pragma unroll
  for (int v = 0; v < VT; ++v) {
    const int c = v * 16 + lg * 4;
    if (c < vdim) {
      float g[4], w[4];
      load4(gate + c, g), load4(p.norm + c, w);
#pragma unroll
      for (int r = 0; r < 4; ++r) g[r] = o[v][r] * rs * w[r] * (g[r] / (1.f + __expf(-g[r])));
      store4(out + c, g);
    }
  }
}

// ---------------------------------------------------------------- host side
#define GLA_MAX_LDS (160 * 1024)
static int gla_lds_out(int dim, int vdim, int e) { return GLA_C * gla_stride(dim) * (4 + e) + gla_dim16(vdim) * GLA_TS * e; }
static int gla_lds_chunk(int dim, int vdim, int e) {
  return GLA_C * gla_stride(dim) * 4 + gla_key_rows(dim) * GLA_TS * 4 + gla_dim16(vdim) * GLA_TS * e;
}

// chunks of a call (0: token by token)
extern "C" int p3v_gla_plan(int B, int L, int H, int dim, int vdim, int f32) {
  if (B <= 0 || L <= 8 || H <= 0 || dim <= 0 || vdim <= 0 || dim % 8 || vdim % 8 || dim > 128 || vdim > 256 || H > 65535 || B > 65535) return 0;
  const int e = f32 ? 4 : 2;
  if (gla_lds_out(dim, vdim, e) > GLA_MAX_LDS || gla_lds_chunk(dim, vdim, e) > GLA_MAX_LDS) return 0;
  return p3v_cdiv(L, GLA_C);
}
extern "C" int64_t p3v_gla_ws_bytes(int B, int L, int H, int dim, int vdim, int n_chunk) {
  if (B <= 0 || L <= 0 || H <= 0 || dim <= 0 || vdim <= 0 || n_chunk < 0) return 0;
  if (n_chunk == 0) return L == 1 ? 0 : (int64_t)B * H * dim * vdim * 4;        // the state behind tokens that do not stay
  return ((int64_t)n_chunk * B * H * ((int64_t)dim * vdim + dim) + (int64_t)B * L * H * dim) * 4;
}

template <typename T> static int gla_steps(const GlaP& p, hipStream_t s) {
  const bool vec = p.vdim % 4 == 0;
  const int nc = vec ? p.vdim / 4 : p.vdim, ng = max(1, 512 / nc);
  const size_t lds = (size_t)(4 * p.dim + p.vdim + ng * p.vdim) * 4;
  if (nc > 512 || lds > 64 * 1024) return P3V_ERR_UNSUPPORTED;
  if (vec) hipLaunchKernelGGL((k_gla_steps<T, 4>), dim3(p.H, p.B), dim3(512), lds, s, p);
  else hipLaunchKernelGGL((k_gla_steps<T, 1>), dim3(p.H, p.B), dim3(512), lds, s, p);
  P3V_CHECK_LAUNCH();
  return P3V_OK;
}
static int gla_set_lds(const void* fn, bool& done) {
  if (!done && hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, GLA_MAX_LDS) != hipSuccess) return P3V_ERR_HIP;
  done = true;
  return P3V_OK;
}
template <typename T, int NK, int NV> static int gla_chunk(const GlaP& p, int nc, hipStream_t s) {
  static bool set = false;
  if (gla_set_lds((const void*)k_gla_chunk<T, NK, NV>, set) != P3V_OK) return P3V_ERR_HIP;
  hipLaunchKernelGGL((k_gla_chunk<T, NK, NV>), dim3(nc, p.H, p.B), dim3(256), gla_lds_chunk(p.dim, p.vdim, (int)sizeof(T)), s, p);
  P3V_CHECK_LAUNCH();
  return P3V_OK;
}
template <typename T, int NK> static int gla_chunk_v(const GlaP& p, int nc, hipStream_t s) {
  return p.vdim <= 64 ? gla_chunk<T, NK, 1>(p, nc, s) : p.vdim <= 128 ? gla_chunk<T, NK, 2>(p, nc, s) : gla_chunk<T, NK, 4>(p, nc, s);
}
template <typename T> static int gla_states(GlaP p, int n_tok, int store, hipStream_t s) {
  const int nc = p3v_cdiv(n_tok, GLA_C);
  p.n_tok = n_tok, p.store = store;
  const int rc = p.dim <= 64 ? gla_chunk_v<T, 1>(p, nc, s) : gla_chunk_v<T, 2>(p, nc, s);
  if (rc != P3V_OK) return rc;
  hipLaunchKernelGGL(k_gla_scan, dim3(p3v_cdiv((long)p.dim * p.vdim / 4, 256), p.B * p.H), dim3(256), 0, s, p, nc);
  P3V_CHECK_LAUNCH();
  return P3V_OK;
}
template <typename T, int VT> static int gla_out(const GlaP& p, int nc, hipStream_t s) {
  static bool set = false;
  if (gla_set_lds((const void*)k_gla_out<T, VT>, set) != P3V_OK) return P3V_ERR_HIP;
  hipLaunchKernelGGL((k_gla_out<T, VT>), dim3(nc, p.H, p.B), dim3(256), gla_lds_out(p.dim, p.vdim, (int)sizeof(T)), s, p);
  P3V_CHECK_LAUNCH();
  return P3V_OK;
}
template <typename T> static int gla_chunks(GlaP p, int nc, hipStream_t s) {
  int rc = gla_states<T>(p, p.L, p.keep == p.L, s);
  if (rc != P3V_OK) return rc;
  p.n_tok = p.L;
  rc = p.vdim <= 32 ? gla_out<T, 2>(p, nc, s) : p.vdim <= 64 ? gla_out<T, 4>(p, nc, s) : p.vdim <= 96 ? gla_out<T, 6>(p, nc, s)
     : p.vdim <= 128 ? gla_out<T, 8>(p, nc, s) : p.vdim <= 192 ? gla_out<T, 12>(p, nc, s) : gla_out<T, 16>(p, nc, s);
  if (rc == P3V_OK && p.keep > 0 && p.keep < p.L) rc = gla_states<T>(p, p.keep, 1, s);      // (the workspace is free again)
  return rc;
}

extern "C" int p3v_gla(const p3v_gla_args_t* a, void* stream) {
  if (!a || !a->y || !a->a2 || !a->a2_b || !a->norm || !a->s || !a->out) return P3V_ERR_ARG;
  if (a->B <= 0 || a->L <= 0 || a->H <= 0 || a->dim <= 0 || a->vdim <= 0 || a->rank <= 0 || a->R < 2 || a->keep < 0 || a->keep > a->L) return P3V_ERR_ARG;
  if (a->ld < 2 * a->H * (a->dim + a->vdim) + a->rank || (!a->d_past && a->past < 0) || a->n_chunk < 0) return P3V_ERR_ARG;
  const GlaP p = {a->y, a->a2, a->a2_b, a->norm, a->s, a->out, a->ws, a->pad_len, a->d_past, a->eps, 1.f / a->tau, a->q_scale,
                  a->B, a->L, a->H, a->dim, a->vdim, a->rank, a->ld, a->past, a->R, a->keep, a->L, 1};
  hipStream_t s = (hipStream_t)stream;
  if (a->n_chunk == 0) {
    if (a->L > 1 && !a->ws) return P3V_ERR_ARG;
    return a->f32 ? gla_steps<float>(p, s) : gla_steps<bf16_t>(p, s);
  }
  if (a->n_chunk != p3v_gla_plan(a->B, a->L, a->H, a->dim, a->vdim, a->f32) || !a->ws || a->ld % 8 || (((uintptr_t)a->y | (uintptr_t)a->ws) & 15)) return P3V_ERR_ARG;
  return a->f32 ? gla_chunks<float>(p, a->n_chunk, s) : gla_chunks<bf16_t>(p, a->n_chunk, s);
}
