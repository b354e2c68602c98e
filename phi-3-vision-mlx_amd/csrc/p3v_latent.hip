// Latent attention: the cache holds one latent c and one rotated key part per token, shared by all heads; per head
//
//   score = scale (q_nope . (uk_h c) + q_rot . k_rot),   out = sum_j p_j (uv_h c_j),   with a sink in the softmax and an output gate.
//
// A few new tokens attend in the latent space -- uk_h is applied to the query, uv_h to the attended latent, so that the cache is read as
// it is, once for 16 heads:
//   k_latent_q      q_nope -> uk_h^T q_nope, rotation of q_rot; one more workgroup norms, rotates and appends the new latent
//   k_latent_attn   16 heads x a run of 64-key tiles, split over the keys
//   k_latent_out    merge of the splits with the sink, uv_h, gate
// Prompts expand keys and values once per call (p3v_latent_prompt.hip).  k_latent_any: any sizes, fp32 arithmetic.
#include "p3v_latent.h"

// ---------------------------------------------------------------- append: one wave per new token
#define LAT_VEC_RANK 1024            // widest latent of the vector form
// latent = rms(c) c_norm, key part rotated -> cache row.  rot_q: the queries of the row are rotated in place, four pairs at a time where V = 4.
template <typename T, int V = 1>
__device__ __forceinline__ void latent_append_row(const LatP& p, int row, int lane, bool rot_q) {
  const int b = row / p.L, past = p.d_past ? *p.d_past : p.past, col = past + row - b * p.L, first = p.pad_len ? p.pad_len[b] : 0;
  const int pos = min(max(col - first, 0), p.tab_n - 1), half = p.rot / 2, W = p.dim + p.rot;
  T* y = (T*)p.y + (size_t)row * p.ld;
  const T* d = y + lat_dkv_col(p);
  T* dst = (T*)p.c + ((size_t)b * p.Tp + col) * (p.rankp + p.rotp);
  const float *cs = p.cos_t + (size_t)pos * half, *sn = p.sin_t + (size_t)pos * half;
  float ss = 0.f;
  if constexpr (V == 4) {                                                // the latent in registers, read once
    float x[LAT_VEC_RANK / 512][8], w[LAT_VEC_RANK / 512][8];
#pragma unroll
    for (int k = 0; k < LAT_VEC_RANK / 512; ++k) {
      const int i = (k * 64 + lane) * 8;
#pragma unroll
      for (int j = 0; j < 8; ++j) x[k][j] = 0.f;
      if (i < p.rank) load_acts<8>(d + i, x[k]), load_acts<8>(p.c_norm + i, w[k]);
#pragma unroll
      for (int j = 0; j < 8; ++j) ss += x[k][j] * x[k][j];
    }
    const float r = 1.f / sqrtf(wave_sum(ss) / (float)p.rank + p.eps);
#pragma unroll
    for (int k = 0; k < LAT_VEC_RANK / 512; ++k) {
      const int i = (k * 64 + lane) * 8;
      if (i < p.rank) {
#pragma unroll
        for (int j = 0; j < 8; ++j) x[k][j] *= r * w[k][j];
        store_acts<8>(dst + i, x[k]);
      }
    }
  } else {
    for (int i = lane; i < p.rank; i += 64) { const float v = load_act(d + i); ss += v * v; }
    const float r = 1.f / sqrtf(wave_sum(ss) / (float)p.rank + p.eps);
    for (int i = lane; i < p.rank; i += 64) store_act(dst + i, load_act(d + i) * r * bf16_to_f32(p.c_norm[i]));
  }
  for (int i = lane; i < half; i += 64) {
    const float u = load_act(d + p.rank + i), v = load_act(d + p.rank + half + i);
    store_act(dst + p.rankp + i, u * cs[i] - v * sn[i]);
    store_act(dst + p.rankp + half + i, v * cs[i] + u * sn[i]);
  }
  if constexpr (V == 4) {
    if (rot_q) {
      const int per = half / 4;
#pragma unroll 2
      for (int e = lane; e < p.H * per; e += 64) {
        const int h = e / per, i = (e - h * per) * 4;
        T* q = y + h * W + p.dim + i;
        float u[4], v[4], c[4], s[4], a[4], b4[4];
        load4(q, u), load4(q + half, v), load4(cs + i, c), load4(sn + i, s);
#pragma unroll
        for (int j = 0; j < 4; ++j) a[j] = u[j] * c[j] - v[j] * s[j], b4[j] = v[j] * c[j] + u[j] * s[j];
        store4(q, a), store4(q + half, b4);
      }
    }
    return;
  }
  if (rot_q)
    for (int e = lane; e < p.H * half; e += 64) {
      const int h = e / half, i = e - h * half;
      T* q = y + h * W + p.dim + i;
      const float u = load_act(q), v = load_act(q + half);
      store_act(q, u * cs[i] - v * sn[i]);
      store_act(q + half, v * cs[i] + u * sn[i]);
    }
}
template <typename T, int V>
__global__ void __launch_bounds__(256) k_latent_append(LatP p) {
  const int row = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (row < p.B * p.L) latent_append_row<T, V>(p, row, threadIdx.x & 63, true);
}

// ---------------------------------------------------------------- queries into the latent space
__global__ void __launch_bounds__(256) k_latent_q(LatP p) {
  const int h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lc = lane & 15, lg = lane >> 4;
  const int row0 = blockIdx.z * 16, M = p.B * p.L, W = p.dim + p.rot, half = p.rot / 2, QW = p.rankp + p.rotp, HP = (p.H + 15) / 16 * 16;
  if (h == p.H) {
    if (blockIdx.y == 0)
      for (int i = wave; i < 16; i += 4)
        if (row0 + i < M) latent_append_row<bf16_t, 4>(p, row0 + i, lane, false);
    return;
  }
  const int r0 = blockIdx.y * 64 + wave * 16, row = min(row0 + lc, M - 1);
  const bf16_t* w = p.ukt + ((size_t)h * p.rankp + r0 + lc) * p.dimp + lg * 8;
  const bf16_t* q = (const bf16_t*)p.y + (size_t)row * p.ld + h * W;
  f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int c = 0; c < p.dimp; c += 32) {
    u32x4_t qv = {0u, 0u, 0u, 0u};
    if (c + lg * 8 < p.dim) qv = *(const u32x4_t*)(q + c + lg * 8);
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8_t*)(w + c), __builtin_bit_cast(bf16x8_t, qv), acc, 0, 0, 0);
  }
  bf16_t* out = (bf16_t*)p.q + ((size_t)(row0 + lc) * HP + h) * QW;
  if (row0 + lc < M) *(u32x2_t*)(out + r0 + lg * 4) = (u32x2_t){pack_bf16x2(acc[0], acc[1]), pack_bf16x2(acc[2], acc[3])};
  if (blockIdx.y == 0) {
    const int past = p.d_past ? *p.d_past : p.past;
    for (int e = tid; e < 16 * half; e += 256) {
      const int m = row0 + e / half, i = e % half;
      if (m >= M) break;
      const int b = m / p.L, pos = min(max(past + m - b * p.L - (p.pad_len ? p.pad_len[b] : 0), 0), p.tab_n - 1);
      const float cs = p.cos_t[(size_t)pos * half + i], sn = p.sin_t[(size_t)pos * half + i];
      const bf16_t* src = (const bf16_t*)p.y + (size_t)m * p.ld + h * W + p.dim + i;
      const float u = bf16_to_f32(src[0]), v = bf16_to_f32(src[half]);
      bf16_t* dst = (bf16_t*)p.q + ((size_t)m * HP + h) * QW + p.rankp + i;
      dst[0] = f32_to_bf16(u * cs - v * sn), dst[half] = f32_to_bf16(v * cs + u * sn);
    }
    for (int e = tid; e < 16 * (p.rotp - p.rot); e += 256) {
      const int m = row0 + e / (p.rotp - p.rot), i = e % (p.rotp - p.rot);
      if (m < M) ((bf16_t*)p.q)[((size_t)m * HP + h) * QW + p.rankp + p.rot + i] = 0;
    }
  }
}

// ---------------------------------------------------------------- attention in the latent space
// 4 waves, 16 heads, tiles of 64 keys.  Wave w holds keys 16 w .. + 15 of a tile as MFMA fragments straight from the cache: the scores come
// from them, and the latent part goes into LDS as rows, from where the value product reads it transposed (ds_read_b64_tr_b16: 16 lanes
// name four rows of 16 elements and receive four rows' values of one column each).  Wave w owns ranks 16 RC w .. of the output.  The next
// tile's fragments are requested as soon as this one's are in LDS.  Partials: (max, sum) pairs, then the unnormalised latents.
__device__ __forceinline__ float* lat_ml(float* ws, const LatP& p, size_t row, int split) { return ws + ((row * p.n_split + split) * p.H) * 2; }
__device__ __forceinline__ float* lat_o(float* ws, const LatP& p, size_t rows, size_t row, int split) {
  return ws + rows * p.n_split * p.H * 2 + (row * p.n_split + split) * p.H * p.rankp;
}
typedef short s16x4_t __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) s16x4_t* tr_ptr_t;
__device__ __forceinline__ u32x2_t lds_read_tr(const bf16_t* at) {
  return __builtin_bit_cast(u32x2_t, __builtin_amdgcn_ds_read_tr16_b64_v4i16((tr_ptr_t)(uintptr_t)(uint32_t)(uintptr_t)at));
}

template <int RC, int RT> struct LatCfg {
  static constexpr int NC = 2 * RC + RT, CS = RC * 64 + 16, QS = NC * 32 + 8, PS = 72;
  static constexpr int TILE = 64 * CS * 2, Q = 16 * QS * 2, P = 16 * PS * 2, LDS = TILE + Q + P + 256;
};
template <int RC, int RT>
__global__ void __launch_bounds__(256) k_latent_attn(LatP p) {
  typedef LatCfg<RC, RT> C;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  bf16_t *tile = (bf16_t*)smem, *Q = (bf16_t*)(smem + C::TILE), *P = (bf16_t*)(smem + C::TILE + C::Q);
  float* red = (float*)(smem + C::TILE + C::Q + C::P);                   // [4][16]
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lc = lane & 15, lg = lane >> 4;
  const int split = blockIdx.x, h0 = blockIdx.y * 16, row = blockIdx.z, b = row / p.L;
  const int QW = p.rankp + p.rotp, HP = (p.H + 15) / 16 * 16, t_first = split * p.tiles_per_split;
  const bf16_t* kb = (const bf16_t*)p.c + ((size_t)b * p.Tp + wave * 16 + lc) * QW + lg * 8;
  bf16x8_t kf[C::NC];
  auto load = [&](int t) {
    const bf16_t* kr = kb + (size_t)t * 64 * QW;
#pragma unroll
    for (int c = 0; c < C::NC; ++c) kf[c] = *(const bf16x8_t*)(kr + c * 32);
  };
  load(min(t_first, (p.Tp >> 6) - 1));                                   // (ahead of the position: the run's first tile, in most calls)
  const int past = p.d_past ? *p.d_past : p.past, pos = past + row - b * p.L, first = p.pad_len ? p.pad_len[b] : 0, last = pos >> 6;
  if (t_first > last) return;                                            // beyond the live keys: the merge does not look here
  const int t0 = max(t_first, first >> 6), t1 = min(t_first + p.tiles_per_split, last + 1), h = h0 + lc;
  float* ml = lat_ml(p.ws, p, row, split);
  if (t0 >= t1) {                                                        // only padding here
    if (tid < 16 && h < p.H) ml[2 * h] = LAT_NEG, ml[2 * h + 1] = 0.f;
    return;
  }
  if (t0 != t_first) load(t0);
  const bf16_t* qg = (const bf16_t*)p.q + ((size_t)row * HP + h0) * QW;
  for (int e = tid; e < 16 * (C::NC * 4); e += 256) {
    const int i = e / (C::NC * 4), c = (e - i * (C::NC * 4)) * 8;
    *(u32x4_t*)(Q + i * C::QS + c) = *(const u32x4_t*)(qg + (size_t)min(i, p.H - 1 - h0) * QW + c);
  }
  f32x4_t o[RC];
#pragma unroll
  for (int j = 0; j < RC; ++j) o[j] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
  const float sc = p.scale * LAT_LOG2E;
  float m_run = LAT_NEG, l_run = 0.f;                                    // of head lc; the sum over this lane's keys
  lds_barrier();
  for (int t = t0; t < t1; ++t) {
    f32x4_t s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int c = 0; c < C::NC; ++c) s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[c], *(const bf16x8_t*)(Q + lc * C::QS + c * 32 + lg * 8), s, 0, 0, 0);
#pragma unroll
    for (int c = 0; c < 2 * RC; ++c) *(bf16x8_t*)(tile + (wave * 16 + lc) * C::CS + c * 32 + lg * 8) = kf[c];
    if (t + 1 < t1) load(t + 1);
    const int key = t * 64 + wave * 16 + lg * 4;
#pragma unroll
    for (int r = 0; r < 4; ++r) s[r] = key + r <= pos && key + r >= first ? s[r] * sc : LAT_NEG;
    const float mx = rows_max(fmaxf(fmaxf(s[0], s[1]), fmaxf(s[2], s[3])));
    if (lg == 0) red[wave * 16 + lc] = mx;
    lds_barrier();
    const float mn = fmaxf(fmaxf(fmaxf(red[lc], red[16 + lc]), fmaxf(red[32 + lc], red[48 + lc])), m_run), al = __builtin_amdgcn_exp2f(m_run - mn);
    float e[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) e[r] = __builtin_amdgcn_exp2f(s[r] - mn);
    l_run = l_run * al + ((e[0] + e[1]) + (e[2] + e[3]));
    m_run = mn;
    *(u32x2_t*)(P + lc * C::PS + wave * 16 + lg * 4) = (u32x2_t){pack_bf16x2(e[0], e[1]), pack_bf16x2(e[2], e[3])};
    lds_barrier();
#pragma unroll
    for (int j = 0; j < RC; ++j) o[j] *= al;
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      const bf16x8_t pf = *(const bf16x8_t*)(P + lc * C::PS + ks * 32 + lg * 8);
      const bf16_t* src = tile + (ks * 32 + lg * 8 + (lc >> 2)) * C::CS + wave * RC * 16 + (lc & 3) * 4;
#pragma unroll
      for (int j = 0; j < RC; ++j) {
        const u32x2_t a = lds_read_tr(src + j * 16), c = lds_read_tr(src + 4 * C::CS + j * 16);
        const u32x4_t v = {a[0], a[1], c[0], c[1]};
        o[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, v), pf, o[j], 0, 0, 0);
      }
    }
    lds_barrier();
  }
  const float l = rows_sum(l_run);
  if (lg == 0) red[wave * 16 + lc] = l;
  lds_barrier();
  if (h >= p.H) return;
  if (wave == 0 && lg == 0) ml[2 * h] = m_run, ml[2 * h + 1] = (red[lc] + red[16 + lc]) + (red[32 + lc] + red[48 + lc]);
  float* od = lat_o(p.ws, p, (size_t)p.B * p.L, row, split) + (size_t)h * p.rankp + wave * RC * 16 + lg * 4;
#pragma unroll
  for (int j = 0; j < RC; ++j) *(float4*)(od + j * 16) = make_float4(o[j][0], o[j][1], o[j][2], o[j][3]);
}

// ---------------------------------------------------------------- merge, value up-projection, gate
// A workgroup per (head, 32 value dimensions, 16 rows): two 16-dimension tiles x four quarters of the rank; weights and, for few rows, the
// partials are requested before anything else.
#define LAT_MAX_SPLIT 128
template <int RC>
__global__ void __launch_bounds__(512) k_latent_out(LatP p) {
  constexpr int OS = RC * 64 + 8;
  __shared__ float wt[16][LAT_MAX_SPLIT];
  __shared__ __attribute__((aligned(16))) bf16_t ol[16 * OS];
  __shared__ float4 part[512];
  const int h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lc = lane & 15, lg = lane >> 4;
  const int row0 = blockIdx.z * 16, M = p.B * p.L, n_row = min(16, M - row0), kq = wave >> 1, v0 = blockIdx.y * 32 + (wave & 1) * 16;
  constexpr int R4 = RC * 16, U = 8;                                     // float4 columns of a latent; splits requested at once
  const int items = n_row * R4, G = items >= 512 ? 1 : 512 / items, g = G > 1 ? tid / items : 0;
  const size_t step = (size_t)p.H * p.rankp;
  auto part_of = [&](int e) { return lat_o(p.ws, p, M, row0 + e / R4, 0) + (size_t)h * p.rankp + 4 * (e % R4); };
  // few rows: the partials are requested before anything else -- which of them were written is known later
  float4 x0[U];
  if (G > 1) {
    const float* o = part_of(tid - g * items);
#pragma unroll
    for (int u = 0; u < U; ++u) x0[u] = *(const float4*)(o + min(min(g, G - 1) + u * G, p.n_split - 1) * step);
  }
  const int past = p.d_past ? *p.d_past : p.past;
  constexpr int NW = (RC + 1) / 2;                                       // 32-rank chunks kq, kq + 4, .. of this wave
  bf16x8_t w[NW];
  const bf16_t* wr = p.uv + ((size_t)h * p.vdim + min(v0 + lc, p.vdim - 1)) * p.rankp + lg * 8;
#pragma unroll
  for (int c = 0; c < NW; ++c) w[c] = *(const bf16x8_t*)(wr + min(kq + 4 * c, 2 * RC - 1) * 32);
  auto live = [&](int row) { return min(p.n_split, ((past + row % p.L) >> 6) / p.tiles_per_split + 1); };
  const float sk = bf16_to_f32(p.sink[h]) * LAT_LOG2E;
  const int v = v0 + lg * 4;
  const u32x2_t z = *(const u32x2_t*)((const bf16_t*)p.y + (size_t)(row0 + min(lc, n_row - 1)) * p.ld + lat_gate_col(p) + h * p.vdim + min(v, p.vdim - 4));
  for (int i = wave; i < n_row; i += 8) {
    const int row = row0 + i, n = live(row);
    float m[2], l[2];
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int s = lane + 64 * j;
      m[j] = LAT_NEG, l[j] = 0.f;
      if (s < n) { const float2 q = *(const float2*)(lat_ml(p.ws, p, row, s) + 2 * h); m[j] = q.x, l[j] = q.y; }
    }
    const float mm = wave_max(fmaxf(fmaxf(m[0], m[1]), sk)), w0 = __builtin_amdgcn_exp2f(m[0] - mm), w1 = __builtin_amdgcn_exp2f(m[1] - mm);
    const float f = 1.f / (wave_sum(l[0] * w0 + l[1] * w1) + __builtin_amdgcn_exp2f(sk - mm));
    wt[i][lane] = m[0] > 0.5f * LAT_NEG ? w0 * f : -1.f;                 // (-1: no such split, or one of padding whose outputs were not written)
    wt[i][lane + 64] = m[1] > 0.5f * LAT_NEG ? w1 * f : -1.f;
  }
  for (int e = tid; e < (16 - n_row) * OS; e += 512) ol[n_row * OS + e] = 0;
  __syncthreads();
  for (int e = G > 1 ? tid - g * items : tid; e < items; e += 512) {
    const int i = e / R4, c = e - i * R4, n = live(row0 + i);
    const float* o = part_of(e);
    float4 a = make_float4(0.f, 0.f, 0.f, 0.f);
    auto add = [&](const float4 (&x)[U], int s0) {
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int s = s0 + u * G;
        const float f = s < n ? wt[i][s] : -1.f;
        if (f >= 0.f) a.x = fmaf(f, x[u].x, a.x), a.y = fmaf(f, x[u].y, a.y), a.z = fmaf(f, x[u].z, a.z), a.w = fmaf(f, x[u].w, a.w);
      }
    };
    if (g < G) {
      if (G > 1) add(x0, g);
      for (int s0 = G > 1 ? g + U * G : g; s0 < n; s0 += U * G) {
        float4 x[U];
#pragma unroll
        for (int u = 0; u < U; ++u) x[u] = *(const float4*)(o + min(s0 + u * G, n - 1) * step);
        add(x, s0);
      }
    }
    if (G == 1) *(u32x2_t*)(ol + i * OS + 4 * c) = (u32x2_t){pack_bf16x2(a.x, a.y), pack_bf16x2(a.z, a.w)};
    else part[tid] = a;
  }
  if (G > 1) {
    __syncthreads();
    if (tid < items) {
      float4 a = part[tid];
      for (int k = 1; k < G; ++k) { const float4 x = part[k * items + tid]; a.x += x.x, a.y += x.y, a.z += x.z, a.w += x.w; }
      const int i = tid / R4, c = tid - i * R4;
      *(u32x2_t*)(ol + i * OS + 4 * c) = (u32x2_t){pack_bf16x2(a.x, a.y), pack_bf16x2(a.z, a.w)};
    }
  }
  __syncthreads();
  f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int c = 0; c < NW; ++c)
    if (kq + 4 * c < 2 * RC) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[c], *(const bf16x8_t*)(ol + lc * OS + (kq + 4 * c) * 32 + lg * 8), acc, 0, 0, 0);
  f32x4_t* sum = (f32x4_t*)part;
  if (kq) sum[tid] = acc;                                                // (nobody reads the merge's use of it any more)
  __syncthreads();
  if (kq == 0 && lc < n_row && v < p.vdim) {
#pragma unroll
    for (int k = 1; k < 4; ++k) acc += sum[tid + 128 * k];
    const size_t row = row0 + lc;
    *(u32x2_t*)((bf16_t*)p.out + row * p.H * p.vdim + h * p.vdim + v) =
        (u32x2_t){pack_bf16x2(acc[0] * lat_gate(bf16lo(z[0])), acc[1] * lat_gate(bf16hi(z[0]))),
                  pack_bf16x2(acc[2] * lat_gate(bf16lo(z[1])), acc[3] * lat_gate(bf16hi(z[1])))};
  }
}

// ---------------------------------------------------------------- any sizes, fp32 arithmetic: a workgroup per (head, row)
#define LAT_ANY_KT 256
template <typename T>
__global__ void __launch_bounds__(256) k_latent_any(LatP p) {
  extern __shared__ float sm[];
  float *ql = sm, *qr = ql + p.rank, *ol = qr + p.rot, *pr = ol + p.rank;       // [rank], [rot], [rank], [KT]
  __shared__ float red[4];
  const int h = blockIdx.x, row = blockIdx.y, b = row / p.L, tid = threadIdx.x;
  const int past = p.d_past ? *p.d_past : p.past, pos = past + row - b * p.L, first = p.pad_len ? p.pad_len[b] : 0, W = p.dim + p.rot;
  const size_t cw = p.rankp + p.rotp;
  const T *y = (const T*)p.y + (size_t)row * p.ld, *q = y + h * W, *c = (const T*)p.c + (size_t)b * p.Tp * cw;
  for (int r = tid; r < p.rank; r += 256) {
    float a = 0.f;
    for (int d = 0; d < p.dim; ++d) a = fmaf(bf16_to_f32(p.uk[((size_t)h * p.dim + d) * p.rankp + r]), load_act(q + d), a);
    ql[r] = a, ol[r] = 0.f;
  }
  for (int i = tid; i < p.rot; i += 256) qr[i] = load_act(q + p.dim + i);
  float m = bf16_to_f32(p.sink[h]), l = 1.f;                     // an online softmax that starts from the sink
  __syncthreads();
  for (int t0 = first; t0 <= pos; t0 += LAT_ANY_KT) {
    const int key = t0 + tid;
    float s = -INFINITY;
    if (key <= pos) {
      const T* k = c + key * cw;
      float a = 0.f;
      for (int r = 0; r < p.rank; ++r) a = fmaf(ql[r], load_act(k + r), a);
      for (int i = 0; i < p.rot; ++i) a = fmaf(qr[i], load_act(k + p.rankp + i), a);
      s = a * p.scale;
    }
    const float mn = fmaxf(m, block_max(s, red)), al = expf(m - mn), e = key <= pos ? expf(s - mn) : 0.f;
    pr[tid] = e;
    l = l * al + block_sum(e, red);                              // (its barriers publish pr)
    m = mn;
    const int n = min(LAT_ANY_KT, pos - t0 + 1);
    for (int r = tid; r < p.rank; r += 256) {
      float a = ol[r] * al;
      for (int j = 0; j < n; ++j) a = fmaf(pr[j], load_act(c + (t0 + j) * cw + r), a);
      ol[r] = a;
    }
    __syncthreads();
  }
  const int lane = tid & 63;
  for (int v = tid >> 6; v < p.vdim; v += 4) {
    const bf16_t* w = p.uv + ((size_t)h * p.vdim + v) * p.rankp;
    float a = 0.f;
    for (int r = lane; r < p.rank; r += 64) a = fmaf(bf16_to_f32(w[r]), ol[r], a);
    a = wave_sum(a);
    if (lane == 0) store_act((T*)p.out + ((size_t)row * p.H + h) * p.vdim + v, a / l * lat_gate(load_act(y + lat_gate_col(p) + h * p.vdim + v)));
  }
}

// ---------------------------------------------------------------- host side
int p3v_latent_check(const p3v_latent_args_t* a) {
  if (!a || !a->y || !a->c_norm || !a->sink || !a->cos_t || !a->sin_t || !a->c) return P3V_ERR_ARG;
  if (a->B <= 0 || a->L <= 0 || a->H <= 0 || a->dim <= 0 || a->rot <= 0 || a->rot % 2 || a->vdim <= 0 || a->rank <= 0) return P3V_ERR_ARG;
  if (a->rankp < a->rank || a->rankp % 64 || a->rotp < a->rot || a->rotp % 32 || a->Tp <= 0 || a->Tp % 64 || a->tab_n <= 0) return P3V_ERR_ARG;
  if (a->ld < a->H * (a->dim + a->rot + a->vdim) + a->rank + a->rot) return P3V_ERR_ARG;
  if (!a->d_past && (a->past < 0 || a->past + a->L > a->Tp || a->past + a->L > a->tab_n)) return P3V_ERR_ARG;
  if ((int64_t)a->B * a->L > 65535 * 16) return P3V_ERR_ARG;
  return P3V_OK;
}
static bool lat_aligned(int dim, int rot, int vdim, int rank) { return dim % 8 == 0 && rot % 8 == 0 && vdim % 8 == 0 && rank % 8 == 0; }
static bool lat_rows_fit(int rank, int rot) { return (rank + 63) / 64 <= 8 && (rot + 31) / 32 <= 2; }

extern "C" int p3v_latent_plan(int B, int L, int H, int dim, int rot, int vdim, int rank, int n_keys, int f32) {
  if (B <= 0 || L <= 0 || H <= 0 || n_keys <= 0 || f32 || !lat_aligned(dim, rot, vdim, rank)) return 0;
  if (L <= 16) {
    if (!lat_rows_fit(rank, rot) || (long)B * L > 65535) return 0;
    const long wgs = (long)p3v_cdiv(H, 16) * B * L;
    const int want = p3v_tuning().mix_wgs, tiles = p3v_cdiv(n_keys, 64);
    const int per = p3v_cdiv(tiles, max(1L, min((long)LAT_MAX_SPLIT, (want > 0 ? want : 256) / wgs)));
    return p3v_cdiv(tiles, per);
  }
  return p3v_latent_prompt_fits(dim, rot, vdim) && B <= 65535 ? -1 : 0;
}
extern "C" int64_t p3v_latent_ws_bytes(int B, int L, int H, int rank, int n_split) {
  if (B <= 0 || L <= 0 || H <= 0 || rank <= 0 || n_split <= 0) return 0;
  return (int64_t)B * L * n_split * H * ((rank + 63) / 64 * 64 + 2) * 4;
}

extern "C" int p3v_latent_append(const p3v_latent_args_t* a, void* stream) {
  const int rc = p3v_latent_check(a);
  if (rc != P3V_OK) return rc;
  const LatP p = lat_params(a);
  const dim3 grid(p3v_cdiv((long)p.B * p.L, 4));
  hipStream_t s = (hipStream_t)stream;
  const bool vec = lat_aligned(p.dim, p.rot, p.vdim, p.rank) && p.ld % 8 == 0 && p.rank <= LAT_VEC_RANK &&
                   (((uintptr_t)p.y | (uintptr_t)p.c | (uintptr_t)p.c_norm | (uintptr_t)p.cos_t | (uintptr_t)p.sin_t) & 15) == 0;
  if (a->f32) {
    if (vec) hipLaunchKernelGGL((k_latent_append<float, 4>), grid, dim3(256), 0, s, p);
    else hipLaunchKernelGGL((k_latent_append<float, 1>), grid, dim3(256), 0, s, p);
  } else {
    if (vec) hipLaunchKernelGGL((k_latent_append<bf16_t, 4>), grid, dim3(256), 0, s, p);
    else hipLaunchKernelGGL((k_latent_append<bf16_t, 1>), grid, dim3(256), 0, s, p);
  }
  P3V_CHECK_LAUNCH();
  return P3V_OK;
}

extern "C" int p3v_latent_any(const p3v_latent_args_t* a, void* stream) {
  const int rc = p3v_latent_check(a);
  if (rc != P3V_OK) return rc;
  if (!a->uk || !a->uv || !a->out) return P3V_ERR_ARG;
  const LatP p = lat_params(a);
  const size_t lds = (size_t)(2 * p.rank + p.rot + LAT_ANY_KT) * 4;
  if (lds > 60 * 1024 || (long)p.B * p.L > 65535) return P3V_ERR_UNSUPPORTED;
  const dim3 grid(p.H, p.B * p.L);
  if (a->f32) hipLaunchKernelGGL(k_latent_any<float>, grid, dim3(256), lds, (hipStream_t)stream, p);
  else hipLaunchKernelGGL(k_latent_any<bf16_t>, grid, dim3(256), lds, (hipStream_t)stream, p);
  P3V_CHECK_LAUNCH();
  return P3V_OK;
}

template <int RC, int RT> static int launch_attn(const LatP& p, hipStream_t s) {
  static bool set = false;
  if (!set) {
    if (hipFuncSetAttribute((const void*)k_latent_attn<RC, RT>, hipFuncAttributeMaxDynamicSharedMemorySize, LatCfg<RC, RT>::LDS) != hipSuccess) return P3V_ERR_HIP;
    set = true;
  }
  hipLaunchKernelGGL((k_latent_attn<RC, RT>), dim3(p.n_split, p3v_cdiv(p.H, 16), p.B * p.L), dim3(256), (LatCfg<RC, RT>::LDS), s, p);
  hipLaunchKernelGGL(k_latent_out<RC>, dim3(p.H, p3v_cdiv(p.vdim, 32), p3v_cdiv(p.B * p.L, 16)), dim3(512), 0, s, p);
  P3V_CHECK_LAUNCH();
  return P3V_OK;
}
template <int RC> static int launch_rows(const LatP& p, hipStream_t s) { return p.rotp == 32 ? launch_attn<RC, 1>(p, s) : launch_attn<RC, 2>(p, s); }

extern "C" int p3v_latent_rows(const p3v_latent_args_t* a, void* stream) {
  const int rc = p3v_latent_check(a);
  if (rc != P3V_OK) return rc;
  if (!a->ukt || !a->uv || !a->q || !a->out || !a->ws || a->n_split <= 0 || a->n_split > LAT_MAX_SPLIT) return P3V_ERR_ARG;
  if (a->f32 || !lat_aligned(a->dim, a->rot, a->vdim, a->rank) || !lat_rows_fit(a->rank, a->rot) || a->ld % 8) return P3V_ERR_UNSUPPORTED;
  if (a->rankp != (a->rank + 63) / 64 * 64 || a->rotp != (a->rot + 31) / 32 * 32 || a->dimp < a->dim || a->dimp % 32) return P3V_ERR_ARG;
  if ((long)a->B * a->L > 65535 || (((uintptr_t)a->y | (uintptr_t)a->ukt | (uintptr_t)a->uv | (uintptr_t)a->c | (uintptr_t)a->c_norm | (uintptr_t)a->q | (uintptr_t)a->ws | (uintptr_t)a->out) & 15)) return P3V_ERR_ARG;
  LatP p = lat_params(a);
  // (the position may be a device value: the splits then cover the capacity)
  p.tiles_per_split = p3v_cdiv(p3v_cdiv(a->L == 1 || a->d_past ? a->Tp : a->past + a->L, 64), a->n_split);
  hipStream_t s = (hipStream_t)stream;
  hipLaunchKernelGGL(k_latent_q, dim3(p.H + 1, p.rankp / 64, p3v_cdiv(p.B * p.L, 16)), dim3(256), 0, s, p);
  P3V_CHECK_LAUNCH();
  switch (p.rankp / 64) {
    case 1: return launch_rows<1>(p, s);
    case 2: return launch_rows<2>(p, s);
    case 3: return launch_rows<3>(p, s);
    case 4: return launch_rows<4>(p, s);
    case 5: return launch_rows<5>(p, s);
    case 6: return launch_rows<6>(p, s);
    case 7: return launch_rows<7>(p, s);
    default: return launch_rows<8>(p, s);
  }
}
