// Gated linear attention: a recurrence with a [dim, vdim] state per head and a decay per key channel,
//
//   S_t = diag(a_t) S_{t-1} + k_t v_t^T,   o_t = S_t^T q_t,   a = sigmoid(W_a2 a1 + b)^(1 / tau),
//
// then an RMS norm of o over vdim and a SiLU gate.  Everything that enters the recurrence is fp32 (the products run on the fp32 matrix
// cores), whatever the activations' type; the states are fp32.
//
// One new token: a workgroup per (head, sequence) reads the state out of the ring's slot past % R and writes the next slot.
// A prompt: chunks of 64 tokens in three launches --
//   k_gla_chunk   per chunk: what its tokens leave in the state, sum_s (k_s a_{s+1} .. a_end) v_s^T, and the whole chunk's decay
//   k_gla_scan    per state element: the states at the chunks' starts, in order
//   k_gla_out     per chunk: (q_t a_1 .. a_t) S_start + sum_{s <= t} (q_t a_{s+1} .. a_t . k_s) v_s, norm, gate
// Decays are kept as running sums of log2 a (c_t); every exponential taken is of c_t - c_s with s <= t, never positive, so that no decay
// is too strong for it: across the 16-token blocks of a chunk both factors refer to the later block's start, inside a block the
// difference is taken pair by pair.
#include "p3v_layered.h"

#define GLA_C 64                     // tokens of a chunk
#define GLA_LOG2E 1.4426950408889634f

struct GlaP {
  const void* y; const bf16_t* a2; const bf16_t* a2b; const bf16_t* norm; float* s; void* out; float* ws;
  const int32_t* pad_len; const int32_t* d_past;
  float eps, inv_tau, q_scale;
  int B, L, H, dim, vdim, rank, ld, past, R, keep, n_tok, store;
};

// log2 of the decay, from z = W_a2 a1 + b
__device__ __forceinline__ float log2_decay(float z, float inv_tau) {
  return (fminf(z, 0.f) - log1pf(expf(-fabsf(z)))) * inv_tau * GLA_LOG2E;
}
__device__ __forceinline__ float row16_sum(float v) {
  v += P3V_DPP_F32(v, 0xB1);
  v += P3V_DPP_F32(v, 0x4E);
  v += P3V_DPP_F32(v, 0x124);
  return v + P3V_DPP_F32(v, 0x128);
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
  float *q = sm, *k = q + dim, *al = k + dim, *v = al + dim, *po = v + vdim;      // po [ng][vdim]
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
      for (int r = 0; r < p.rank; ++r) z = fmaf(bf16_to_f32(w[r]), load_act(a1 + r), z);
      al[d] = __builtin_amdgcn_exp2f(log2_decay(z, p.inv_tau));
    }
    for (int i = tid; i < vdim; i += 512) v[i] = load_act(row + 2 * p.H * dim + h * vdim + i);
    __syncthreads();
    if (mine) {
      float o[V], vv[V];
#pragma unroll
      for (int j = 0; j < V; ++j) o[j] = 0.f, vv[j] = v[c + j];
      auto update = [&](int d, float (&x)[V]) {
        const float a = al[d], kd = k[d], qd = q[d];
#pragma unroll
        for (int j = 0; j < V; ++j) {
          x[j] = live ? fmaf(a, x[j], kd * vv[j]) : 0.f;
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
// c[t][d] (row stride S) = sum of log2 a over the chunk's tokens up to t, 256 threads.  a1: LDS scratch of 64 x 17 floats.  Tokens that
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
    __syncthreads();
    for (int i = tid; i < GLA_C * 16; i += 256) {
      const int t = i >> 4, r = i & 15;
      a1[t * 17 + r] = t >= lo && t < hi && r < nr ? load_act(base + (size_t)t * p.ld + r0 + r) : 0.f;
    }
    __syncthreads();
    if (mine) {
      float w[16];
#pragma unroll
      for (int r = 0; r < 16; ++r) w[r] = r < nr ? bf16_to_f32(p.a2[(size_t)(h * dim + d) * p.rank + r0 + r]) : 0.f;
      const float bias = bf16_to_f32(p.a2b[h * dim + d]);
      for (int t = g * per; t < (g + 1) * per; ++t) {
        float z = r0 == 0 ? bias : c[t * S + d];
#pragma unroll
        for (int r = 0; r < 16; ++r) z = fmaf(w[r], a1[t * 17 + r], z);
        c[t * S + d] = z;
      }
    }
  }
  if (mine) {
    float run = 0.f;
    for (int t = g * per; t < (g + 1) * per; ++t) {
      if (t >= lo && t < hi) run += log2_decay(c[t * S + d], p.inv_tau);
      c[t * S + d] = run;
    }
  }
  __syncthreads();
  float off = 0.f;
  if (mine)
    for (int i = 0; i < g; ++i) off += c[((i + 1) * per - 1) * S + d];
  __syncthreads();
  if (mine && g > 0)
    for (int t = g * per; t < (g + 1) * per; ++t) c[t * S + d] += off;
  __syncthreads();
}
// the live tokens [lo, hi) of a chunk
__device__ __forceinline__ void gla_span(const GlaP& p, int b, int l0, int& lo, int& hi) {
  const int past = p.d_past ? *p.d_past : p.past, first = p.pad_len ? p.pad_len[b] : 0;
  lo = min(max(first - past - l0, 0), GLA_C);
  hi = max(min(p.n_tok - l0, GLA_C), lo);
}
__host__ __device__ __forceinline__ int gla_stride1(int n) { return (n + 63) / 64 * 64 + 16; }   // four rows of 16 floats in distinct banks
__host__ __device__ __forceinline__ int gla_stride(int n) { return (n + 7) / 8 * 8 + 4; }        // sixteen rows of 4 floats in distinct banks

__host__ __device__ __forceinline__ size_t gla_decay_at(const GlaP& p, int nc) { return (size_t)nc * p.B * p.H * p.dim * p.vdim; }

template <typename T>
__global__ void __launch_bounds__(256) k_gla_chunk(GlaP p) {
  extern __shared__ float sm[];
  const int ch = blockIdx.x, h = blockIdx.y, b = blockIdx.z, tid = threadIdx.x, lane = tid & 63, lc = lane & 15, lg = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int dim = p.dim, vdim = p.vdim, KS = gla_stride1(dim), VS = gla_stride1(vdim), l0 = ch * GLA_C;
  float *kd = sm, *v = kd + GLA_C * KS, *a1 = v;                 // (the values come when the decays are done)
  int lo, hi;
  gla_span(p, b, l0, lo, hi);
  gla_decays<T>(p, b, h, l0, lo, hi, kd, KS, a1);
  const T* base = (const T*)p.y + ((size_t)b * p.L + l0) * p.ld;
  for (int i = tid; i < GLA_C * (vdim / 8); i += 256) {
    const int t = i / (vdim / 8), c = (i - t * (vdim / 8)) * 8;
    float x[8] = {0, 0, 0, 0, 0, 0, 0, 0};
    if (t >= lo && t < hi) load_acts<8>(base + (size_t)t * p.ld + 2 * p.H * dim + h * vdim + c, x);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[t * VS + c + j] = x[j];
  }
  const size_t row = (size_t)ch * p.B * p.H + (size_t)b * p.H + h;
  float* decay = p.ws + gla_decay_at(p, gridDim.x) + row * dim;
  float end[8];                                                  // this thread's 8 channels at the chunk's end
  const int per = dim / 8, c8 = (tid % per) * 8, t8 = tid / per, nt = 256 / per;
#pragma unroll
  for (int j = 0; j < 8; ++j) end[j] = kd[(GLA_C - 1) * KS + c8 + j];
  if (t8 == 0)
#pragma unroll
    for (int j = 0; j < 8; ++j) decay[c8 + j] = __builtin_amdgcn_exp2f(end[j]);
  __syncthreads();
  if (t8 < nt)
    for (int t = t8; t < GLA_C; t += nt) {
      float x[8] = {0, 0, 0, 0, 0, 0, 0, 0};
      if (t >= lo && t < hi) load_acts<8>(base + (size_t)t * p.ld + (p.H + h) * dim + c8, x);
#pragma unroll
      for (int j = 0; j < 8; ++j) kd[t * KS + c8 + j] = x[j] * __builtin_amdgcn_exp2f(fminf(end[j] - kd[t * KS + c8 + j], 0.f));
    }
  __syncthreads();
  // A operand: row = key channel, k = token; B operand: column = value channel
  const int dt = (dim + 15) / 16, vg = (vdim + 63) / 64;
  float* dst = p.ws + row * dim * vdim;
  for (int u = wave; u < dt * vg; u += 4) {
    const int d0 = (u / vg) * 16, v0 = (u % vg) * 64;
    f32x4_t acc[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
    const float* ka = kd + lg * KS + d0 + lc;
    const float* va = v + lg * VS + v0 + lc;
#pragma unroll 4
    for (int s = 0; s < GLA_C; s += 4) {
      const float a = ka[s * KS];
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, va[s * VS + j * 16], acc[j], 0, 0, 0);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = d0 + lg * 4 + r, c = v0 + j * 16 + lc;
        if (d < dim && c < vdim) dst[(size_t)d * vdim + c] = acc[j][r];
      }
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

// Wave w owns the chunk's tokens 16 w .. 16 w + 15; VG: groups of 64 value channels.
template <typename T> struct GlaOutLds {
  int DS, VS, PS, cum, k, qt, v, p, total;                       // strides (elements) and byte offsets
  __host__ __device__ GlaOutLds(int dim, int vdim) {
    DS = gla_stride(dim), VS = (vdim + 15) / 16 * 16 + 8, PS = GLA_C + 4;
    cum = 0, qt = cum + GLA_C * DS * 4, p = qt + GLA_C * DS * 4, k = p + GLA_C * PS * 4, v = k + GLA_C * DS * (int)sizeof(T);
    total = v + GLA_C * VS * (int)sizeof(T);
  }
};
template <typename T, int VG>
__global__ void __launch_bounds__(256) k_gla_out(GlaP p) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  const int ch = blockIdx.x, h = blockIdx.y, b = blockIdx.z, tid = threadIdx.x, lane = tid & 63, lc = lane & 15, lg = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int dim = p.dim, vdim = p.vdim, l0 = ch * GLA_C;
  const GlaOutLds<T> o_(dim, vdim);
  const int DS = o_.DS, VS = o_.VS, PS = o_.PS;
  float *cum = (float*)(smem + o_.cum), *qt = (float*)(smem + o_.qt), *P = (float*)(smem + o_.p);
  T *k = (T*)(smem + o_.k), *v = (T*)(smem + o_.v);
  int lo, hi;
  gla_span(p, b, l0, lo, hi);
  gla_decays<T>(p, b, h, l0, lo, hi, cum, DS, P);
  const T* base = (const T*)p.y + ((size_t)b * p.L + l0) * p.ld;
  for (int i = tid; i < GLA_C * (dim / 4); i += 256) {           // (4 at a time: the strides are multiples of 4)
    const int t = i / (dim / 4), c = (i - t * (dim / 4)) * 4;
    const bool live = t >= lo && t < hi;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      k[t * DS + c + j] = live ? base[(size_t)t * p.ld + (p.H + h) * dim + c + j] : (T)0;
      qt[t * DS + c + j] = live ? load_act(base + (size_t)t * p.ld + h * dim + c + j) * p.q_scale : 0.f;
    }
  }
  for (int i = tid; i < GLA_C * (vdim / 4); i += 256) {
    const int t = i / (vdim / 4), c = (i - t * (vdim / 4)) * 4;
    const bool live = t >= lo && t < hi;
#pragma unroll
    for (int j = 0; j < 4; ++j) v[t * VS + c + j] = live ? base[(size_t)t * p.ld + 2 * p.H * dim + h * vdim + c + j] : (T)0;
  }
  __syncthreads();
  const int t0 = wave * 16;

  // ---- the block's own pairs: lane = (token s, quarter of the channels), all 16 tokens t
  {
    float sc[16];
#pragma unroll
    for (int t = 0; t < 16; ++t) sc[t] = 0.f;
    for (int d = lg; d < dim; d += 4) {
      const float ks = load_act(k + (t0 + lc) * DS + d), cs = cum[(t0 + lc) * DS + d];
#pragma unroll
      for (int t = 0; t < 16; ++t)
        sc[t] = fmaf(qt[(t0 + t) * DS + d] * ks, __builtin_amdgcn_exp2f(fminf(cum[(t0 + t) * DS + d] - cs, 0.f)), sc[t]);
    }
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      const float x = rows_sum(sc[t]);
      if (lg == (t >> 2)) P[(t0 + t) * PS + t0 + lc] = t >= lc ? x : 0.f;
    }
  }
  // ---- earlier blocks of the chunk: both factors refer to the block's start
  const float* ref = cum + max(t0 - 1, 0) * DS;                  // (wave 0: the chunk's start, zero)
  for (int i = lane; i < 16 * dim; i += 64) {
    const int t = t0 + i / dim, d = i % dim;
    qt[t * DS + d] *= __builtin_amdgcn_exp2f(fminf(cum[t * DS + d] - (wave ? ref[d] : 0.f), 0.f));
  }
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");             // (the wave's own rows: no barrier)
  const float* qa = qt + (t0 + lc) * DS + lg;
  if (wave) {
    f32x4_t sc[3];
#pragma unroll
    for (int j = 0; j < 3; ++j) sc[j] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
    for (int d0 = 0; d0 < dim; d0 += 4) {
      const float a = qa[d0], rd = ref[d0 + lg];
#pragma unroll
      for (int j = 0; j < 3; ++j)
        if (j < wave) {
          const int s = j * 16 + lc;
          const float kb = load_act(k + s * DS + d0 + lg) * __builtin_amdgcn_exp2f(fminf(rd - cum[s * DS + d0 + lg], 0.f));
          sc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, kb, sc[j], 0, 0, 0);
        }
    }
#pragma unroll
    for (int j = 0; j < 3; ++j)
      if (j < wave) {
#pragma unroll
        for (int r = 0; r < 4; ++r) P[(t0 + lg * 4 + r) * PS + j * 16 + lc] = sc[j][r];
      }
  }
  // ---- the state at the chunk's start, then the pairs
  f32x4_t o[VG][4];
#pragma unroll
  for (int g = 0; g < VG; ++g)
#pragma unroll
    for (int j = 0; j < 4; ++j) o[g][j] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
  const float* S = p.ws + ((size_t)ch * p.B * p.H + (size_t)b * p.H + h) * dim * vdim;
  int vc[VG][4];
#pragma unroll
  for (int g = 0; g < VG; ++g)
#pragma unroll
    for (int j = 0; j < 4; ++j) vc[g][j] = min(g * 64 + j * 16 + lc, vdim - 1);
#pragma unroll 2
  for (int d0 = 0; d0 < dim; d0 += 4) {
    const float a = wave ? qa[d0] * __builtin_amdgcn_exp2f(ref[d0 + lg]) : qa[d0];
    const float* sr = S + (size_t)(d0 + lg) * vdim;
#pragma unroll
    for (int g = 0; g < VG; ++g)
#pragma unroll
      for (int j = 0; j < 4; ++j) o[g][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, sr[vc[g][j]], o[g][j], 0, 0, 0);
  }
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  const float* pa = P + (t0 + lc) * PS + lg;
#pragma unroll 2
  for (int s = 0; s < t0 + 16; s += 4) {
    const float a = pa[s];
    const T* vr = v + (s + lg) * VS;
#pragma unroll
    for (int g = 0; g < VG; ++g)
#pragma unroll
      for (int j = 0; j < 4; ++j) o[g][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, load_act(vr + vc[g][j]), o[g][j], 0, 0, 0);
  }
  // ---- norm over the value channels (a token: 4 registers rows x 16 lanes), gate
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    float ss = 0.f;
#pragma unroll
    for (int g = 0; g < VG; ++g)
#pragma unroll
      for (int j = 0; j < 4; ++j) ss += g * 64 + j * 16 + lc < vdim ? o[g][j][r] * o[g][j][r] : 0.f;
    const float rs = 1.f / sqrtf(row16_sum(ss) / (float)vdim + p.eps);
    const int t = t0 + lg * 4 + r, l = l0 + t;
    if (l >= p.L) continue;
    const T* gate = base + (size_t)t * p.ld + 2 * p.H * dim + (p.H + h) * vdim;
    T* out = (T*)p.out + ((size_t)b * p.L + l) * p.H * vdim + (size_t)h * vdim;
#pragma unroll
    for (int g = 0; g < VG; ++g)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int c = g * 64 + j * 16 + lc;
        if (c < vdim) store_act(out + c, o[g][j][r] * rs * bf16_to_f32(p.norm[c]) * silu32(load_act(gate + c)));
      }
  }
}

// ---------------------------------------------------------------- host side
#define GLA_MAX_LDS (160 * 1024)
static int gla_lds_out(int dim, int vdim, int f32) { return f32 ? GlaOutLds<float>(dim, vdim).total : GlaOutLds<bf16_t>(dim, vdim).total; }
static int gla_lds_chunk(int dim, int vdim) { return GLA_C * (gla_stride1(dim) + max(gla_stride1(vdim), 17)) * 4; }

// chunks of a call (0: token by token)
extern "C" int p3v_gla_plan(int B, int L, int H, int dim, int vdim, int f32) {
  if (B <= 0 || L <= 8 || H <= 0 || dim <= 0 || vdim <= 0 || dim % 8 || vdim % 8 || dim > 128 || vdim > 256 || H > 65535 || B > 65535) return 0;
  if (gla_lds_out(dim, vdim, f32) > GLA_MAX_LDS || gla_lds_chunk(dim, vdim) > GLA_MAX_LDS) return 0;
  return p3v_cdiv(L, GLA_C);
}
extern "C" int64_t p3v_gla_ws_bytes(int B, int L, int H, int dim, int vdim, int n_chunk) {
  if (B <= 0 || L <= 0 || H <= 0 || dim <= 0 || vdim <= 0 || n_chunk < 0) return 0;
  if (n_chunk == 0) return L == 1 ? 0 : (int64_t)B * H * dim * vdim * 4;        // the state behind tokens that do not stay
  return (int64_t)n_chunk * B * H * ((int64_t)dim * vdim + dim) * 4;
}

template <typename T> static int gla_steps(const GlaP& p, hipStream_t s) {
  const bool vec = p.vdim % 4 == 0;
  const int nc = vec ? p.vdim / 4 : p.vdim, ng = max(1, 512 / nc);
  const size_t lds = (size_t)(3 * p.dim + p.vdim + ng * p.vdim) * 4;
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
template <typename T> static int gla_states(GlaP p, int n_tok, int store, hipStream_t s) {
  static bool set = false;
  if (gla_set_lds((const void*)k_gla_chunk<T>, set) != P3V_OK) return P3V_ERR_HIP;
  const int nc = p3v_cdiv(n_tok, GLA_C);
  p.n_tok = n_tok, p.store = store;
  hipLaunchKernelGGL(k_gla_chunk<T>, dim3(nc, p.H, p.B), dim3(256), gla_lds_chunk(p.dim, p.vdim), s, p);
  hipLaunchKernelGGL(k_gla_scan, dim3(p3v_cdiv((long)p.dim * p.vdim / 4, 256), p.B * p.H), dim3(256), 0, s, p, nc);
  P3V_CHECK_LAUNCH();
  return P3V_OK;
}
template <typename T, int VG> static int gla_out(const GlaP& p, int nc, hipStream_t s) {
  static bool set = false;
  if (gla_set_lds((const void*)k_gla_out<T, VG>, set) != P3V_OK) return P3V_ERR_HIP;
  hipLaunchKernelGGL((k_gla_out<T, VG>), dim3(nc, p.H, p.B), dim3(256), GlaOutLds<T>(p.dim, p.vdim).total, s, p);
  P3V_CHECK_LAUNCH();
  return P3V_OK;
}
template <typename T> static int gla_chunks(GlaP p, int nc, hipStream_t s) {
  int rc = gla_states<T>(p, p.L, p.keep == p.L, s);
  if (rc != P3V_OK) return rc;
  p.n_tok = p.L;
  rc = p.vdim <= 64 ? gla_out<T, 1>(p, nc, s) : p.vdim <= 128 ? gla_out<T, 2>(p, nc, s) : gla_out<T, 4>(p, nc, s);
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
