// Row kernels and plain projections of the layered text decoders (config.py: LayerSpec): a residual stream in fp32, RMS norms and
// dynamic-tanh "norms" of it, token shift, whole-projection query / key norms, value mixing, and a projection for every size and for
// fp32 activations.
// Activations are bf16 or fp32 (the element type T of a model); weights are bf16 in either case, which fp32 arithmetic reads exactly.
#include "p3v_layered.h"

// ---------------------------------------------------------------- x = table[id] * scale, fp32
__global__ void __launch_bounds__(256) k_embed_scale(const int32_t* __restrict__ ids, const bf16_t* __restrict__ table, float* __restrict__ out,
                                                     int hidden, int vocab, float scale) {
  const int t = blockIdx.x;
  int id = ids[t];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  for (int c = threadIdx.x; c < hidden; c += 256) out[(size_t)t * hidden + c] = bf16_to_f32(table[(size_t)id * hidden + c]) * scale;
}

extern "C" int p3v_embed_scale(const int32_t* ids, const uint16_t* table, float* out, int n_tok, int hidden, int vocab, float scale,
                               void* stream) {
  if (!ids || !table || !out || n_tok < 0 || hidden <= 0 || vocab <= 0) return P3V_ERR_ARG;
  if (n_tok == 0) return P3V_OK;
  hipLaunchKernelGGL(k_embed_scale, dim3(n_tok), dim3(256), 0, (hipStream_t)stream, ids, table, out, hidden, vocab, scale);
  P3V_CHECK_LAUNCH();
  return P3V_OK;
}

// ---------------------------------------------------------------- RMS norm of fp32 rows
// out = x / sqrt(mean x^2 + eps) * w * gain, fp32 up to the one rounding of out; a wave per row, CH 16-byte chunks per lane in registers
// (CH = 0: any width, the row read twice)
template <typename T, int CH>
__global__ void __launch_bounds__(256) k_rms_rows(const float* __restrict__ x, const bf16_t* __restrict__ w, T* __restrict__ out, int rows, int H,
                                                  float eps, float gain) {
  const int row = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (row >= rows) return;
  const float* xr = x + (size_t)row * H;
  T* o = out + (size_t)row * H;
  float ss = 0.f;
  if constexpr (CH > 0) {
    const int chunks = H / 8;
    float v[CH][8];
    u32x4_t g[CH];
#pragma unroll
    for (int i = 0; i < CH; ++i) {
      const int c = min(i * 64 + lane, chunks - 1);
      load_acts<8>(xr + 8 * c, v[i]);
      g[i] = *(const u32x4_t*)(w + 8 * c);
    }
#pragma unroll
    for (int i = 0; i < CH; ++i)
      if (i * 64 + lane < chunks) {
#pragma unroll
        for (int j = 0; j < 8; ++j) ss += v[i][j] * v[i][j];
      }
    const float r = gain / sqrtf(wave_sum(ss) / (float)H + eps);
#pragma unroll
    for (int i = 0; i < CH; ++i)
      if (i * 64 + lane < chunks) {
#pragma unroll
        for (int j = 0; j < 8; ++j) v[i][j] *= r * (j & 1 ? bf16hi(g[i][j >> 1]) : bf16lo(g[i][j >> 1]));
        store_acts<8>(o + 8 * (i * 64 + lane), v[i]);
      }
  } else {
    for (int c = lane; c < H; c += 64) ss += xr[c] * xr[c];
    const float r = gain / sqrtf(wave_sum(ss) / (float)H + eps);
    for (int c = lane; c < H; c += 64) store_act(o + c, xr[c] * (r * bf16_to_f32(w[c])));
  }
}
template <typename T>
static void launch_rms_rows(const float* x, const bf16_t* w, T* out, int rows, int H, float eps, float gain, hipStream_t s) {
  const dim3 grid(p3v_cdiv(rows, 4));
  if (H % 8 || (((uintptr_t)x | (uintptr_t)w | (uintptr_t)out) & 15) || H > 4096) hipLaunchKernelGGL((k_rms_rows<T, 0>), grid, dim3(256), 0, s, x, w, out, rows, H, eps, gain);
  else if (H <= 1024) hipLaunchKernelGGL((k_rms_rows<T, 2>), grid, dim3(256), 0, s, x, w, out, rows, H, eps, gain);
  else if (H <= 2048) hipLaunchKernelGGL((k_rms_rows<T, 4>), grid, dim3(256), 0, s, x, w, out, rows, H, eps, gain);
  else hipLaunchKernelGGL((k_rms_rows<T, 8>), grid, dim3(256), 0, s, x, w, out, rows, H, eps, gain);
}
extern "C" int p3v_rms_rows(const float* x, const uint16_t* w, void* out, int out_f32, int rows, int H, float eps, float gain, void* stream) {
  if (!x || !w || !out || rows < 0 || H <= 0) return P3V_ERR_ARG;
  if (rows == 0) return P3V_OK;
  if (out_f32) launch_rms_rows(x, w, (float*)out, rows, H, eps, gain, (hipStream_t)stream);
  else launch_rms_rows(x, w, (bf16_t*)out, rows, H, eps, gain, (hipStream_t)stream);
  P3V_CHECK_LAUNCH();
  return P3V_OK;
}

// ---------------------------------------------------------------- dynamic tanh (+ token shift)
// A workgroup takes DYT_ROWS consecutive tokens of one sequence and 256 channels: the unshifted value of the token before is a
// register of the same thread, recomputed only for the first token of the run.
#define DYT_ROWS 8
template <typename T>
__global__ void __launch_bounds__(256) k_dyt(DytP p, T* __restrict__ out, bool store_hist) {
  const int c = blockIdx.x * 256 + threadIdx.x, b = blockIdx.z, l0 = blockIdx.y * DYT_ROWS;
  if (c >= p.H) return;
  const float w = bf16_to_f32(p.w[c]), bb = bf16_to_f32(p.b[c]);
  const float* x = p.x + (size_t)b * p.L * p.H + c;
  const int l1 = min(p.L, l0 + DYT_ROWS);
  if (!p.mu) {
    for (int l = l0; l < l1; ++l) store_act(out + ((size_t)b * p.L + l) * p.H + c, tanhf(x[(size_t)l * p.H] * p.alpha) * w + bb);
    return;
  }
  const int past = p.d_past ? *p.d_past : p.past, first = p.pad_len ? p.pad_len[b] : 0;
  const float mu = bf16_to_f32(p.mu[c]);
  float prev = 0.f;
  if (past + l0 > first)
    prev = l0 > 0 ? tanhf(x[(size_t)(l0 - 1) * p.H] * p.alpha) * w + bb : p.hist[((size_t)b * p.R + (past - 1) % p.R) * p.H + c];
  for (int l = l0; l < l1; ++l) {
    if (past + l == first) prev = 0.f;
    const float h = tanhf(x[(size_t)l * p.H] * p.alpha) * w + bb;
    store_act(out + ((size_t)b * p.L + l) * p.H + c, h + (prev - h) * mu);
    if (store_hist && l >= p.L - p.R) p.hist[((size_t)b * p.R + (past + l) % p.R) * p.H + c] = h;
    prev = h;
  }
}
// the history of a call so long that it wraps onto the slot its own first token reads: a launch of its own, behind k_dyt
__global__ void __launch_bounds__(256) k_dyt_hist(DytP p) {
  const int c = blockIdx.x * 256 + threadIdx.x, b = blockIdx.z, l = p.L - 1 - blockIdx.y;
  if (c >= p.H || l < 0) return;
  const int past = p.d_past ? *p.d_past : p.past;
  p.hist[((size_t)b * p.R + (past + l) % p.R) * p.H + c] = tanhf(p.x[((size_t)b * p.L + l) * p.H + c] * p.alpha) * bf16_to_f32(p.w[c]) + bf16_to_f32(p.b[c]);
}

int p3v_dyt_check(const p3v_dyt_args_t* a) {
  if (!a || !a->x || !a->w || !a->b || a->B <= 0 || a->L <= 0 || a->H <= 0) return P3V_ERR_ARG;
  if (a->mu && (!a->hist || a->hist_rows < 2 || (!a->d_past && a->past < 0))) return P3V_ERR_ARG;
  return P3V_OK;
}

extern "C" int p3v_dyt(const p3v_dyt_args_t* a, void* out, int out_f32, void* stream) {
  const int rc = p3v_dyt_check(a);
  if (rc != P3V_OK || !out) return rc != P3V_OK ? rc : P3V_ERR_ARG;
  const DytP p = dyt_params(a);
  hipStream_t s = (hipStream_t)stream;
  const dim3 grid(p3v_cdiv(p.H, 256), p3v_cdiv(p.L, DYT_ROWS), p.B);
  const bool late = p.mu && p.L >= p.R;
  if (out_f32) hipLaunchKernelGGL(k_dyt<float>, grid, dim3(256), 0, s, p, (float*)out, !late);
  else hipLaunchKernelGGL(k_dyt<bf16_t>, grid, dim3(256), 0, s, p, (bf16_t*)out, !late);
  if (late) hipLaunchKernelGGL(k_dyt_hist, dim3(p3v_cdiv(p.H, 256), p.R, p.B), dim3(256), 0, s, p);
  P3V_CHECK_LAUNCH();
  return P3V_OK;
}

// ---------------------------------------------------------------- projection of any size, fp32 arithmetic
// out[M, N] = A[M, K] W[N, K]^T with plain fp32 FMAs: what an fp32 model runs everywhere (no reduced-precision matrix mode), and
// what a bf16 model runs where a size does not fit the matrix-core kernels.  64 x 64 x 16 tile, 4 x 4 outputs per thread.
struct GemmAnyP {
  const void* A; const bf16_t* W; void* out; const void* resid; const bf16_t* col_scale;
  int M, N, K, lda, ldw, ldo;
};
template <typename T, int EPI>
__global__ void __launch_bounds__(256) k_gemm_any(GemmAnyP p) {
  constexpr bool SILU = P3V_GATED(EPI);
  __shared__ float sa[16][68], sw[SILU ? 2 : 1][16][68];
  const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4, n0 = blockIdx.x * 64, m0 = blockIdx.y * 64;
  const int lr = tid >> 2, lk = (tid & 3) * 4;
  const T* A = (const T*)p.A;
  float acc[SILU ? 2 : 1][4][4] = {};
  for (int k0 = 0; k0 < p.K; k0 += 16) {
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int k = k0 + lk + j;
      sa[lk + j][lr] = (m0 + lr < p.M && k < p.K) ? load_act(A + (size_t)(m0 + lr) * p.lda + k) : 0.f;
#pragma unroll
      for (int u = 0; u < (SILU ? 2 : 1); ++u)
        sw[u][lk + j][lr] = (n0 + lr < p.N && k < p.K) ? bf16_to_f32(p.W[(size_t)(n0 + lr + u * p.N) * p.ldw + k]) : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < 16; ++k) {
      float a[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) a[i] = sa[k][ty * 4 + i];
#pragma unroll
      for (int u = 0; u < (SILU ? 2 : 1); ++u)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float w = sw[u][k][tx * 4 + j];
#pragma unroll
          for (int i = 0; i < 4; ++i) acc[u][i][j] = fmaf(a[i], w, acc[u][i][j]);
        }
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int m = m0 + ty * 4 + i, n = n0 + tx * 4 + j;
      if (m >= p.M || n >= p.N) continue;
      const size_t o = (size_t)m * p.ldo + n;
      const float v = acc[0][i][j];
      if (EPI == P3V_EPI_GELU_MUL) {
        const float t = 1.5957691216057308f * (v + 0.044715f * v * v * v);
        store_act((T*)p.out + o, v / (1.f + expf(-t)) * acc[SILU ? 1 : 0][i][j]);
      } else if (SILU) {
        const float g = round_act<T>(v), u = round_act<T>(acc[SILU ? 1 : 0][i][j]);
        store_act((T*)p.out + o, round_act<T>(g * round_act<T>(1.f / (1.f + expf(-g)))) * u);
      } else if (EPI == P3V_EPI_SCALE_RESID_F32) {
        ((float*)p.out)[o] = ((const float*)p.resid)[o] + bf16_to_f32(p.col_scale[n]) * v;
      } else if (EPI == P3V_EPI_F32) {
        ((float*)p.out)[o] = v;
      } else {
        store_act((T*)p.out + o, v);
      }
    }
}

extern "C" int p3v_gemm_any(const p3v_gemm_args_t* a, int a_f32, void* stream) {
  if (!a || !a->A || !a->W || !a->out || a->M < 0 || a->N <= 0 || a->K <= 0 || a->lda < a->K || a->ldw < a->K || a->ldo < a->N) return P3V_ERR_ARG;
  if (a->epilogue == P3V_EPI_SCALE_RESID_F32 && (!a->resid || !a->col_scale)) return P3V_ERR_ARG;
  if (a->M == 0) return P3V_OK;
  const GemmAnyP p = {a->A, a->W, a->out, a->resid, a->col_scale, a->M, a->N, a->K, a->lda, a->ldw, a->ldo};
  const dim3 grid(p3v_cdiv(a->N, 64), p3v_cdiv(a->M, 64));
  hipStream_t s = (hipStream_t)stream;
#define P3V_ANY(EPI)                                                                                   \
  case EPI:                                                                                            \
    if (a_f32) hipLaunchKernelGGL((k_gemm_any<float, EPI>), grid, dim3(256), 0, s, p);                 \
    else hipLaunchKernelGGL((k_gemm_any<bf16_t, EPI>), grid, dim3(256), 0, s, p);                      \
    break;
  switch (a->epilogue) {
    P3V_ANY(P3V_EPI_NONE)
    P3V_ANY(P3V_EPI_F32)
    P3V_ANY(P3V_EPI_SILU_MUL)
    P3V_ANY(P3V_EPI_GELU_MUL)
    P3V_ANY(P3V_EPI_SCALE_RESID_F32)
    default: return P3V_ERR_UNSUPPORTED;
  }
#undef P3V_ANY
  P3V_CHECK_LAUNCH();
  return P3V_OK;
}

// ---------------------------------------------------------------- head split: whole-projection q / k norms, value mixing, cache append
// gridDim.x walks the 16-token blocks of the value cache that a call touches; gridDim.z shares a block's work: 4 workgroups for the
// query / key norms (a wave per token), 4 for a quarter of the value columns each.
template <typename T, int V>
__global__ void __launch_bounds__(256) k_qkv_heads(QkvHeadsP p) {
  const int b = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int past = p.d_past ? *p.d_past : p.past;
  const int blk = (past >> 4) + blockIdx.x, pos_lo = max(past, blk * 16), pos_hi = min(past + p.L, blk * 16 + 16);
  const int nq = p.H * p.dim, nk = p.G * p.dim, nv = p.G * p.vdim;
  const T* base = (const T*)p.qkv;
  const int part = blockIdx.z;
  const int pos = blk * 16 + part * 4 + wave;
  if (part < 4 && pos >= pos_lo && pos < pos_hi) {
    const int l = pos - past;
    const T* row = base + ((size_t)b * p.L + l) * p.ld;
    float sq = 0.f, sk = 0.f;
    for (int e = lane * V; e < nq; e += 64 * V) { float v[V]; load_acts<V>(row + e, v);
#pragma unroll
      for (int j = 0; j < V; ++j) sq += v[j] * v[j]; }
    for (int e = lane * V; e < nk; e += 64 * V) { float v[V]; load_acts<V>(row + nq + e, v);
#pragma unroll
      for (int j = 0; j < V; ++j) sk += v[j] * v[j]; }
    const float rq = 1.f / sqrtf(wave_sum(sq) / (float)nq + p.eps), rk = 1.f / sqrtf(wave_sum(sk) / (float)nk + p.eps);
    for (int e = lane * V; e < nq; e += 64 * V) {
      const int h = e / p.dim, d = e - h * p.dim;
      float v[V];
      load_acts<V>(row + e, v);
#pragma unroll
      for (int j = 0; j < V; ++j) v[j] = v[j] * rq * bf16_to_f32(p.q_norm[e + j]);
      store_acts<V>((T*)p.q + (((size_t)b * p.H + h) * p.L + l) * p.dimp + d, v);
    }
    for (int e = lane * V; e < nk; e += 64 * V) {
      const int g = e / p.dim, d = e - g * p.dim;
      float v[V];
      load_acts<V>(row + nq + e, v);
#pragma unroll
      for (int j = 0; j < V; ++j) v[j] = v[j] * rk * bf16_to_f32(p.k_norm[e + j]);
      store_acts<V>((T*)p.k + (((size_t)b * p.G + g) * p.Tp + pos) * p.dimp + d, v);
    }
  }
  if (part < 4) return;
  if constexpr (V == 8) {
    // a whole block of 16 tokens: 8 columns per thread, 16-byte loads, the 16 x 8 values turned around in registers
    if (p.vdim % 8 == 0 && (!p.v_first || p.ld_first % 8 == 0) && pos_hi - pos_lo == 16) {
      for (int e = ((part - 4) * 256 + threadIdx.x) * 8; e < nv; e += 8192) {
        const int g = e / p.vdim, d = e - g * p.vdim;
        T* dst = (T*)p.v + ((((size_t)b * p.G + g) * (p.Tp >> 4) + blk) * p.vdimp + d) * 16;
        const T* src = base + ((size_t)b * p.L + pos_lo - past) * p.ld + nq + nk + e;
        const T* first = p.v_first ? (const T*)p.v_first + ((size_t)b * p.L + pos_lo - past) * p.ld_first + e : nullptr;
#pragma unroll
        for (int half = 0; half < 2; ++half) {
          float x[8][8];
#pragma unroll
          for (int j = 0; j < 8; ++j) {
            load_acts<8>(src + (size_t)(half * 8 + j) * p.ld, x[j]);
            if (first) {
              float f[8];
              load_acts<8>(first + (size_t)(half * 8 + j) * p.ld_first, f);
#pragma unroll
              for (int k = 0; k < 8; ++k) x[j][k] = (1.f - p.vmix) * x[j][k] + p.vmix * f[k];
            }
          }
#pragma unroll
          for (int k = 0; k < 8; ++k) {
            float y[8];
#pragma unroll
            for (int j = 0; j < 8; ++j) y[j] = x[j][k];
            store_acts<8>(dst + k * 16 + half * 8, y);
          }
        }
      }
      return;
    }
  }
  for (int e = (part - 4) * 256 + threadIdx.x; e < nv; e += 1024) {
    const int g = e / p.vdim, d = e - g * p.vdim;
    T* dst = (T*)p.v + ((((size_t)b * p.G + g) * (p.Tp >> 4) + blk) * p.vdimp + d) * 16;
    const T* src = base + ((size_t)b * p.L - past) * p.ld + nq + nk + e;            // + pos * ld
    const T* first = p.v_first ? (const T*)p.v_first + ((size_t)b * p.L - past) * p.ld_first + e : nullptr;
    auto value = [&](int pos) {
      const float own = load_act(src + (size_t)pos * p.ld);
      return first ? (1.f - p.vmix) * own + p.vmix * load_act(first + (size_t)pos * p.ld_first) : own;
    };
    if (pos_hi - pos_lo == 16) {
      float v[16];
#pragma unroll
      for (int j = 0; j < 16; ++j) v[j] = value(pos_lo + j);
      store_acts<8>(dst, v);
      store_acts<8>(dst + 8, v + 8);
    } else {
      for (int pos = pos_lo; pos < pos_hi; ++pos) store_act(dst + (pos & 15), value(pos));
    }
  }
}

extern "C" int p3v_qkv_heads(const p3v_mix_args_t* a, void* stream) {
  const int rc = p3v_mix_check(a);
  if (rc != P3V_OK) return rc;
  if (!a->qkv || !a->q || !a->q_norm || !a->k_norm) return P3V_ERR_ARG;
  const QkvHeadsP p = {a->qkv, a->q_norm, a->k_norm, a->v_first, a->q, a->k, a->v, a->d_past, a->eps, a->vmix,
                       a->B, a->L, a->H, a->G, a->dim, a->vdim, a->dimp, a->vdimp, a->ld, a->ld_first, a->past, a->Tp};
  const dim3 grid(a->L == 1 ? 1 : p3v_cdiv(a->L + 15, 16) + (a->d_past ? 1 : 0), a->B, 8);
  const bool vec = a->dim % 8 == 0 && a->ld % 8 == 0;
  hipStream_t s = (hipStream_t)stream;
  if (a->f32) {
    if (vec) hipLaunchKernelGGL((k_qkv_heads<float, 8>), grid, dim3(256), 0, s, p);
    else hipLaunchKernelGGL((k_qkv_heads<float, 1>), grid, dim3(256), 0, s, p);
  } else {
    if (vec) hipLaunchKernelGGL((k_qkv_heads<bf16_t, 8>), grid, dim3(256), 0, s, p);
    else hipLaunchKernelGGL((k_qkv_heads<bf16_t, 1>), grid, dim3(256), 0, s, p);
  }
  P3V_CHECK_LAUNCH();
  return P3V_OK;
}

// ---------------------------------------------------------------- attention with mixed heads, any sizes, fp32 arithmetic
// One workgroup per query row.  Raw scores of ALL heads against 32 keys, mixed across the heads, then an online softmax that starts
// from the sink (m = sink, l = 1).  The plain form of the kernels in p3v_attn_mix.hip; fp32 models and unusual sizes run it.
#define ANY_KT 32
template <typename T>
__global__ void __launch_bounds__(256) k_attn_mix_any(AttnMixP p) {
  extern __shared__ float sm[];
  const int l = blockIdx.x, b = blockIdx.y, tid = threadIdx.x, per = p.H / p.G;
  float* q = sm;                                     // [H][dim]
  float* raw = q + p.H * p.dim;                      // [H][KT]
  float* pr = raw + p.H * ANY_KT;                    // [H][KT]
  float* o = pr + p.H * ANY_KT;                      // [H * vdim]
  float* talk = o + p.H * p.vdim;                    // [H][H]
  float* ms = talk + p.H * p.H;                      // [H] running max
  float* ls = ms + p.H;                              // [H] running sum
  float* al = ls + p.H;                              // [H] rescale factor of this tile
  const int past = p.d_past ? *p.d_past : p.past, pos = past + l, first = p.pad_len ? p.pad_len[b] : 0;
  for (int i = tid; i < p.H * p.dim; i += 256) {
    const int h = i / p.dim, d = i - h * p.dim;
    q[i] = load_act((const T*)p.q + (((size_t)b * p.H + h) * p.L + l) * p.dimp + d);
  }
  for (int i = tid; i < p.H * p.H; i += 256) talk[i] = bf16_to_f32(p.talk[i]);
  for (int i = tid; i < p.H * p.vdim; i += 256) o[i] = 0.f;
  for (int i = tid; i < p.H; i += 256) ms[i] = bf16_to_f32(p.sink[i]), ls[i] = 1.f;
  __syncthreads();
  for (int t0 = first / ANY_KT * ANY_KT; t0 <= pos; t0 += ANY_KT) {
    for (int i = tid; i < p.H * ANY_KT; i += 256) {
      const int h = i / ANY_KT, key = t0 + i % ANY_KT;
      float s = 0.f;
      if (key >= first && key <= pos) {
        const T* kr = (const T*)p.k + (((size_t)b * p.G + h / per) * p.Tp + key) * p.dimp;
        for (int d = 0; d < p.dim; ++d) s = fmaf(q[h * p.dim + d], load_act(kr + d), s);
      }
      raw[i] = s * p.scale;
    }
    __syncthreads();
    for (int i = tid; i < p.H * ANY_KT; i += 256) {
      const int h = i / ANY_KT, j = i % ANY_KT, key = t0 + j;
      float s = 0.f;
      for (int g = 0; g < p.H; ++g) s = fmaf(talk[h * p.H + g], raw[g * ANY_KT + j], s);
      pr[i] = key >= first && key <= pos ? s : -INFINITY;
    }
    __syncthreads();
    for (int h = tid; h < p.H; h += 256) {
      float m = ms[h];
      for (int j = 0; j < ANY_KT; ++j) m = fmaxf(m, pr[h * ANY_KT + j]);
      const float a = expf(ms[h] - m);
      float l_ = ls[h] * a;
      for (int j = 0; j < ANY_KT; ++j) {
        const float e = expf(pr[h * ANY_KT + j] - m);
        pr[h * ANY_KT + j] = e;
        l_ += e;
      }
      ms[h] = m, ls[h] = l_, al[h] = a;
    }
    __syncthreads();
    for (int i = tid; i < p.H * p.vdim; i += 256) {
      const int h = i / p.vdim, d = i - h * p.vdim;
      float acc = o[i] * al[h];
      const int j0 = max(0, first - t0), j1 = min(ANY_KT, pos - t0 + 1);
      for (int j = j0; j < j1; ++j) {
        const int key = t0 + j;
        acc = fmaf(pr[h * ANY_KT + j],
                   load_act((const T*)p.v + ((((size_t)b * p.G + h / per) * (p.Tp >> 4) + (key >> 4)) * p.vdimp + d) * 16 + (key & 15)), acc);
      }
      o[i] = acc;
    }
    __syncthreads();
  }
  const T* gate = (const T*)p.gate + ((size_t)b * p.L + l) * p.ld;
  for (int i = tid; i < p.H * p.vdim; i += 256) {
    const int h = i / p.vdim;
    store_act((T*)p.out + ((size_t)b * p.L + l) * p.H * p.vdim + i, o[i] / ls[h] * (1.f / (1.f + expf(-load_act(gate + h)))));
  }
}

int p3v_mix_check(const p3v_mix_args_t* a) {
  if (!a || !a->k || !a->v || a->B <= 0 || a->L <= 0 || a->H <= 0 || a->G <= 0 || a->H % a->G || a->dim <= 0 || a->vdim <= 0) return P3V_ERR_ARG;
  if (a->dimp < a->dim || a->dimp % 32 || a->vdimp < a->vdim || a->vdimp % 32 || a->Tp <= 0 || a->Tp % 32) return P3V_ERR_ARG;
  if (!a->d_past && (a->past < 0 || a->past + a->L > a->Tp)) return P3V_ERR_ARG;
  return P3V_OK;
}

int p3v_attn_mix_any(const p3v_mix_args_t* a, hipStream_t s) {
  const AttnMixP p = attn_mix_params(a);
  const size_t lds = sizeof(float) * ((size_t)p.H * p.dim + 2 * (size_t)p.H * ANY_KT + (size_t)p.H * p.vdim + (size_t)p.H * p.H + 3 * (size_t)p.H);
  if (lds > 160 * 1024) return P3V_ERR_UNSUPPORTED;
  static bool attr_set = false;
  if (!attr_set) {
    if (hipFuncSetAttribute((const void*)k_attn_mix_any<float>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024) != hipSuccess ||
        hipFuncSetAttribute((const void*)k_attn_mix_any<bf16_t>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024) != hipSuccess)
      return P3V_ERR_HIP;
    attr_set = true;
  }
  const dim3 grid(a->L, a->B);
  if (a->f32) hipLaunchKernelGGL(k_attn_mix_any<float>, grid, dim3(256), lds, s, p);
  else hipLaunchKernelGGL(k_attn_mix_any<bf16_t>, grid, dim3(256), lds, s, p);
  P3V_CHECK_LAUNCH();
  return P3V_OK;
}
