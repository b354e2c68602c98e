// Attention whose heads' scores are mixed before the softmax (score_h <- sum_g talk[h, g] score_g), with a per-head sink in the
// denominator and a per-head output gate.  The mixing couples ALL heads at every (query, key) pair, so a workgroup owns all heads of
// its queries (one head per workgroup, the usual split, would recompute every head's scores in every workgroup).
//
//   K cache [B, G, Tp, dimp]            rows of keys: a row is an MFMA fragment (dimp: dim rounded up to 32, zeros behind)
//   V cache [B, G, Tp / 16, vdimp, 16]  blocks of 16 keys, value dimension by value dimension: the PV product reads 8 consecutive
//                                       keys of one dimension per lane (16 bytes, whole 512-byte runs per wave) and a 16-key tile of
//                                       the decode step is contiguous (vdimp: vdim rounded up to 16)
//
// Scores, their mixing and the softmax are fp32.  The mixing runs on the bf16 matrix cores WITHOUT losing fp32: talk is bf16 data, and
// a score is split into three bf16 terms whose sum is the fp32 value, so that every product is exact and only the fp32 accumulation
// rounds -- an eighth of the cost of the fp32 matrix instruction.
#include "p3v_layered.h"

#define MIX_NEG (-1e30f)             // "no key yet": finite, so that differences of two of them stay 0
#define MIX_MAX_H 32
#define LOG2E 1.4426950408889634f

typedef __attribute__((ext_vector_type(2))) float f32x2_t;

__device__ __forceinline__ float row16_max(float v) {
  v = fmaxf(v, P3V_DPP_F32(v, 0xB1));
  v = fmaxf(v, P3V_DPP_F32(v, 0x4E));
  v = fmaxf(v, P3V_DPP_F32(v, 0x124));
  return fmaxf(v, P3V_DPP_F32(v, 0x128));
}
__device__ __forceinline__ float row16_sum(float v) {
  v += P3V_DPP_F32(v, 0xB1);
  v += P3V_DPP_F32(v, 0x4E);
  v += P3V_DPP_F32(v, 0x124);
  return v + P3V_DPP_F32(v, 0x128);
}
__device__ __forceinline__ float gate_of(const bf16_t* logit) { return 1.f / (1.f + __expf(-bf16_to_f32(*logit))); }

// partials of a split: (max, sum) pairs, then the unnormalised outputs
__device__ __forceinline__ float* ws_ml(float* ws, const AttnMixP& p, size_t row, int split) { return ws + ((row * p.n_split + split) * p.H) * 2; }
__device__ __forceinline__ float* ws_o(float* ws, const AttnMixP& p, size_t rows, size_t row, int split) {
  return ws + rows * p.n_split * p.H * 2 + (row * p.n_split + split) * p.H * p.vdim;
}

// ================================================================ prompts
// 8 waves, 16 queries x all heads, tiles of 32 keys.  Wave w owns heads w * HW .. + HW - 1 in the two matrix products (its Q fragments
// and output accumulators stay in registers, K / V fragments come straight from the cache: no other wave of the workgroup needs
// them) and queries 2w, 2w + 1 of ALL heads in the mixing and the softmax; the two views meet in LDS:
//   S  [16 q][32 keys][heads] fp32 (+ padding: both the writes of HW heads and the reads of 8 heads per lane are conflict-free)
//   P  [heads][16 q][32 keys] bf16,  AL [heads][16 q] rescale factors
template <int HW> struct MixCfg {
  static constexpr int HP = 8 * HW, HS = HP + 4, QS = 32 * HS + 4;      // heads padded, S strides (floats): key, query
  static constexpr int PQ = 40, PH = 16 * PQ + 8;                        // P strides (bf16): query, head
  static constexpr int HM = (HP + 15) / 16;                              // 16-head row blocks of the mixing
  static constexpr int S_BYTES = 16 * QS * 4, P_BYTES = HP * PH * 2, A_BYTES = HP * 16 * 4;
  static constexpr int LDS = S_BYTES + P_BYTES + 2 * A_BYTES;
};

template <int HW, int DC>
__global__ void __launch_bounds__(512, 1) k_attn_mix_prefill(AttnMixP p) {
  typedef MixCfg<HW> C;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  float* S = (float*)smem;
  bf16_t* P = (bf16_t*)(smem + C::S_BYTES);
  float* AL = (float*)(smem + C::S_BYTES + C::P_BYTES);
  float* LS = AL + C::HP * 16;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lc = lane & 15, lg = lane >> 4;
  const int n_qt = (p.L + 15) >> 4, qt = n_qt - 1 - (int)blockIdx.x, split = blockIdx.y, b = blockIdx.z;   // longest rows first
  const int q0 = qt * 16, per = p.H / p.G, past = p.d_past ? *p.d_past : p.past, first = p.pad_len ? p.pad_len[b] : 0;
  const int last = past + min(q0 + 15, p.L - 1);                         // last key any query of the tile sees
  const int t_lo = first >> 5, t_hi = (last >> 5) + 1;
  const int chunk = max(1, (t_hi - t_lo + p.n_split - 1) / p.n_split);
  const int t0 = t_lo + split * chunk, t1 = min(t_hi, t0 + chunk);
  const int dc = p.dimp >> 5, nvt = p.vdimp >> 4;
  const float sc = p.scale * LOG2E;

  // Q fragments (B operand: column = query, 8 consecutive dimensions)
  bf16x8_t qf[HW][DC];
#pragma unroll
  for (int i = 0; i < HW; ++i) {
    const int h = min(wave * HW + i, p.H - 1);
    const bf16_t* qr = (const bf16_t*)p.q + (((size_t)b * p.H + h) * p.L + min(q0 + lc, p.L - 1)) * p.dimp + lg * 8;
#pragma unroll
    for (int c = 0; c < DC; ++c) qf[i][c] = *(const bf16x8_t*)(qr + (c < dc ? c : 0) * 32);
  }
  // talk fragments (A operand: row = mixed head, 8 consecutive raw heads), zero beyond H
  bf16x8_t tf[C::HM];
#pragma unroll
  for (int m = 0; m < C::HM; ++m) {
    u32x4_t w = {0u, 0u, 0u, 0u};
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int h = m * 16 + lc, g = lg * 8 + j;
      const uint32_t v = h < p.H && g < p.H ? p.talk[h * p.H + g] : 0;
      w[j >> 1] |= v << (16 * (j & 1));
    }
    tf[m] = __builtin_bit_cast(bf16x8_t, w);
  }
  f32x4_t o[HW][2 * DC];
#pragma unroll
  for (int i = 0; i < HW; ++i)
#pragma unroll
    for (int d = 0; d < 2 * DC; ++d) o[i][d] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
  float mr[2][C::HM][4], lr[2][C::HM][4];                                // running max / per-lane sum of (query 2w + qi, head 16 m + 4 lg + r)
#pragma unroll
  for (int qi = 0; qi < 2; ++qi)
#pragma unroll
    for (int m = 0; m < C::HM; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) mr[qi][m][r] = MIX_NEG, lr[qi][m][r] = 0.f;

  const bf16_t* kb = (const bf16_t*)p.k + (size_t)b * p.G * p.Tp * p.dimp + (size_t)lc * p.dimp + lg * 8;
  const bf16_t* vb = (const bf16_t*)p.v + (size_t)b * p.G * p.Tp * p.vdimp + ((size_t)(lg >> 1) * p.vdimp + lc) * 16 + (lg & 1) * 8;
  const bool active = wave * HW < p.H;

  for (int t = t0; t < t1; ++t) {
    // ---- raw scores of this wave's heads -> S
    if (active) {
      f32x4_t s[HW][2];
#pragma unroll
      for (int i = 0; i < HW; ++i) s[i][0] = s[i][1] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
      bf16x8_t kf[2][DC];
#pragma unroll
      for (int i = 0; i < HW; ++i) {
        const int h = min(wave * HW + i, p.H - 1), g = h / per;
        if (i == 0 || g != min(wave * HW + i - 1, p.H - 1) / per) {
          const bf16_t* kr = kb + ((size_t)g * p.Tp + t * 32) * p.dimp;
#pragma unroll
          for (int c = 0; c < DC; ++c)
            if (c < dc) {
              kf[0][c] = *(const bf16x8_t*)(kr + c * 32);
              kf[1][c] = *(const bf16x8_t*)(kr + (size_t)16 * p.dimp + c * 32);
            }
        }
#pragma unroll
        for (int c = 0; c < DC; ++c)
          if (c < dc) {
            s[i][0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[0][c], qf[i][c], s[i][0], 0, 0, 0);
            s[i][1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[1][c], qf[i][c], s[i][1], 0, 0, 0);
          }
      }
#pragma unroll
      for (int kt = 0; kt < 2; ++kt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          float* dst = S + lc * C::QS + (kt * 16 + lg * 4 + r) * C::HS + wave * HW;
          if constexpr (HW == 4) *(float4*)dst = make_float4(s[0][kt][r], s[1][kt][r], s[2][kt][r], s[3][kt][r]);
          else if constexpr (HW == 2) *(f32x2_t*)dst = (f32x2_t){s[0][kt][r], s[1][kt][r]};
          else *dst = s[0][kt][r];
        }
    }
    __syncthreads();

    // ---- mixing + softmax of queries 2w, 2w + 1, all heads
#pragma unroll
    for (int qi = 0; qi < 2; ++qi) {
      const int q = 2 * wave + qi, qpos = past + q0 + q;
      f32x4_t mx[C::HM][2];
#pragma unroll
      for (int kt = 0; kt < 2; ++kt) {
        float v[8];
        const float* src = S + q * C::QS + (kt * 16 + lc) * C::HS + lg * 8;
        if (lg * 8 < C::HP) {
          const float4 a = *(const float4*)src, c = *(const float4*)(src + 4);
          v[0] = a.x, v[1] = a.y, v[2] = a.z, v[3] = a.w, v[4] = c.x, v[5] = c.y, v[6] = c.z, v[7] = c.w;
        } else {
#pragma unroll
          for (int j = 0; j < 8; ++j) v[j] = 0.f;
        }
        if (p.H < C::HP) {                                               // (heads that no wave wrote)
#pragma unroll
          for (int j = 0; j < 8; ++j) v[j] = lg * 8 + j < p.H ? v[j] : 0.f;
        }
        u32x4_t part[3];
#pragma unroll
        for (int k = 0; k < 3; ++k)
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const uint32_t pk = pack_bf16x2(v[2 * j], v[2 * j + 1]);
            part[k][j] = pk;
            if (k < 2) v[2 * j] -= bf16lo(pk), v[2 * j + 1] -= bf16hi(pk);
          }
#pragma unroll
        for (int m = 0; m < C::HM; ++m) {
          f32x4_t a = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int k = 2; k >= 0; --k) a = __builtin_amdgcn_mfma_f32_16x16x32_bf16(tf[m], __builtin_bit_cast(bf16x8_t, part[k]), a, 0, 0, 0);
          mx[m][kt] = a;
        }
      }
      const int key0 = t * 32 + lc, key1 = key0 + 16;
      const bool live0 = key0 <= qpos && key0 >= first, live1 = key1 <= qpos && key1 >= first;
#pragma unroll
      for (int m = 0; m < C::HM; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float s0 = live0 ? mx[m][0][r] * sc : -INFINITY, s1 = live1 ? mx[m][1][r] * sc : -INFINITY;
          const float mn = fmaxf(mr[qi][m][r], row16_max(fmaxf(s0, s1)));
          const float al = __builtin_amdgcn_exp2f(mr[qi][m][r] - mn), p0 = __builtin_amdgcn_exp2f(s0 - mn), p1 = __builtin_amdgcn_exp2f(s1 - mn);
          mr[qi][m][r] = mn;
          lr[qi][m][r] = lr[qi][m][r] * al + (p0 + p1);
          const int h = m * 16 + lg * 4 + r;
          if (h < C::HP) {
            bf16_t* dst = P + h * C::PH + q * C::PQ + lc;
            dst[0] = f32_to_bf16(p0), dst[16] = f32_to_bf16(p1);
            if (lc == 0) AL[h * 16 + q] = al;
          }
        }
    }
    __syncthreads();

    // ---- O^T += V^T P^T of this wave's heads
    if (active) {
      bf16x8_t vf[2 * DC];
#pragma unroll
      for (int i = 0; i < HW; ++i) {
        const int h = min(wave * HW + i, p.H - 1), g = h / per;
        if (i == 0 || g != min(wave * HW + i - 1, p.H - 1) / per) {
          const bf16_t* vr = vb + ((size_t)g * (p.Tp >> 4) + t * 2) * p.vdimp * 16;
#pragma unroll
          for (int d = 0; d < 2 * DC; ++d)
            if (d < nvt) vf[d] = *(const bf16x8_t*)(vr + d * 256);
        }
        const bf16x8_t pf = *(const bf16x8_t*)(P + h * C::PH + lc * C::PQ + lg * 8);
        const float al = AL[h * 16 + lc];
#pragma unroll
        for (int d = 0; d < 2 * DC; ++d)
          if (d < nvt) {
            o[i][d] *= al;
            o[i][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[d], pf, o[i][d], 0, 0, 0);
          }
      }
    }
  }

  // ---- the softmax side hands its sums (and maxima) to the head side
#pragma unroll
  for (int qi = 0; qi < 2; ++qi)
#pragma unroll
    for (int m = 0; m < C::HM; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int h = m * 16 + lg * 4 + r;
        const float l = row16_sum(lr[qi][m][r]);
        if (lc == 0 && h < C::HP) LS[h * 16 + 2 * wave + qi] = l;
      }
  __syncthreads();                                                       // (AL of the last tile has been read by every wave)
#pragma unroll
  for (int qi = 0; qi < 2; ++qi)
#pragma unroll
    for (int m = 0; m < C::HM; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int h = m * 16 + lg * 4 + r;
        if (lc == 0 && h < C::HP) AL[h * 16 + 2 * wave + qi] = mr[qi][m][r];
      }
  __syncthreads();
  const int row_q = q0 + lc;
  if (!active || row_q >= p.L) return;
  const size_t row = (size_t)b * p.L + row_q, rows = (size_t)p.B * p.L;
#pragma unroll
  for (int i = 0; i < HW; ++i) {
    const int h = wave * HW + i;
    if (h >= p.H) continue;
    const float m = AL[h * 16 + lc], l = LS[h * 16 + lc];
    float f = 1.f;
    if (p.n_split == 1) {
      const float sk = bf16_to_f32(p.sink[h]) * LOG2E, mm = fmaxf(m, sk);
      f = __builtin_amdgcn_exp2f(m - mm) / (l * __builtin_amdgcn_exp2f(m - mm) + __builtin_amdgcn_exp2f(sk - mm)) * gate_of((const bf16_t*)p.gate + row * p.ld + h);
    } else if (lg == 0) {
      *(f32x2_t*)(ws_ml(p.ws, p, row, split) + h * 2) = (f32x2_t){m, l};
    }
#pragma unroll
    for (int d = 0; d < 2 * DC; ++d)
      if (d < nvt) {
        const int dd = d * 16 + lg * 4;
        if (p.n_split == 1) {
          bf16_t* dst = (bf16_t*)p.out + row * p.H * p.vdim + (size_t)h * p.vdim + dd;
          if (p.vdim % 4 == 0) {
            if (dd < p.vdim) *(u32x2_t*)dst = (u32x2_t){pack_bf16x2(o[i][d][0] * f, o[i][d][1] * f), pack_bf16x2(o[i][d][2] * f, o[i][d][3] * f)};
          } else {
#pragma unroll
            for (int r = 0; r < 4; ++r)
              if (dd + r < p.vdim) dst[r] = f32_to_bf16(o[i][d][r] * f);
          }
        } else {
          float* dst = ws_o(p.ws, p, rows, row, split) + (size_t)h * p.vdim + dd;
#pragma unroll
          for (int r = 0; r < 4; ++r)
            if (dd + r < p.vdim) dst[r] = o[i][d][r];
        }
      }
  }
}

// ================================================================ one new token per sequence
// A workgroup takes a run of 16-key tiles of one sequence, all heads: the query's whole-projection norm is recomputed in every
// workgroup (a few KB), the workgroup whose run holds the new position also normalises and appends the new key and mixes and appends
// the new value.  Partials of the runs are merged by k_attn_mix_combine.
template <int DC, int NP>
__global__ void __launch_bounds__(512) k_attn_mix_decode(QkvHeadsP hp, AttnMixP p) {
  constexpr int SS = 20;                                                 // S / P row stride (floats)
  __shared__ float S[MIX_MAX_H * SS], P[MIX_MAX_H * SS], talk[MIX_MAX_H * (MIX_MAX_H + 1)], AL[MIX_MAX_H], red[16];
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  bf16_t* qs = (bf16_t*)smem;                                            // [H][dimp] normalised query
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lc = lane & 15, lg = lane >> 4;
  const int split = blockIdx.x, b = blockIdx.y, per = p.H / p.G;
  const int past = p.d_past ? *p.d_past : p.past, first = p.pad_len ? p.pad_len[b] : 0;
  const int t_first = split * p.tiles_per_split, own = past >> 4;
  if (t_first > own) return;                                             // beyond the live keys: the merge does not look here
  const int t_begin = max(t_first, first >> 4), t_end = min(t_first + p.tiles_per_split, own + 1);
  const bool owner = own < t_end;
  const int nq = p.H * p.dim, nk = p.G * p.dim, nv = p.G * p.vdim;
  const bf16_t* row = (const bf16_t*)hp.qkv + (size_t)b * hp.ld;
  float* ml = ws_ml(p.ws, p, b, split);
  if (t_begin >= t_end) {                                                // only padding here (and the new position is in no such run)
    for (int h = tid; h < p.H; h += 512) ml[2 * h] = MIX_NEG, ml[2 * h + 1] = 0.f;
    if (!owner) return;                                                  // an idle batch row still appends: its cache stays finite
  }

  // ---- query (and key) norm
  float sq = 0.f, sk = 0.f;
  for (int e = tid; e < nq; e += 512) { const float v = bf16_to_f32(row[e]); sq += v * v; }
  if (owner)
    for (int e = tid; e < nk; e += 512) { const float v = bf16_to_f32(row[nq + e]); sk += v * v; }
  for (int e = tid; e < p.H * p.H; e += 512) { const int h = e / p.H; talk[h * (MIX_MAX_H + 1) + e - h * p.H] = bf16_to_f32(p.talk[e]); }
  const float rq = 1.f / sqrtf(block_sum(sq, red) / (float)nq + hp.eps), rk = 1.f / sqrtf(block_sum(sk, red) / (float)nk + hp.eps);
  for (int e = tid; e < p.H * p.dimp; e += 512) {
    const int h = e / p.dimp, d = e - h * p.dimp;
    qs[e] = d < p.dim ? f32_to_bf16(bf16_to_f32(row[h * p.dim + d]) * rq * bf16_to_f32(hp.q_norm[h * p.dim + d])) : (bf16_t)0;
  }
  if (owner) {
    for (int e = tid; e < nk; e += 512) {
      const int g = e / p.dim, d = e - g * p.dim;
      ((bf16_t*)hp.k)[(((size_t)b * p.G + g) * p.Tp + past) * p.dimp + d] = f32_to_bf16(bf16_to_f32(row[nq + e]) * rk * bf16_to_f32(hp.k_norm[e]));
    }
    for (int e = tid; e < nv; e += 512) {
      const int g = e / p.vdim, d = e - g * p.vdim;
      float v = bf16_to_f32(row[nq + nk + e]);
      if (hp.v_first) v = (1.f - hp.vmix) * v + hp.vmix * bf16_to_f32(((const bf16_t*)hp.v_first)[(size_t)b * hp.ld_first + e]);
      ((bf16_t*)hp.v)[((((size_t)b * p.G + g) * (p.Tp >> 4) + own) * p.vdimp + d) * 16 + (past & 15)] = f32_to_bf16(v);
    }
  }
  __syncthreads();                                                       // the query is in LDS, the new key / value in the cache
  if (t_begin >= t_end) return;

  const int dc = p.dimp >> 5, gw = (p.G + 7) >> 3;                       // kv heads per wave
  const float sc = p.scale * LOG2E;
  const bf16_t* kb = (const bf16_t*)p.k + ((size_t)b * p.G * p.Tp + lc) * p.dimp + lg * 8;
  float acc[NP];
#pragma unroll
  for (int j = 0; j < NP; ++j) acc[j] = 0.f;
  float m_run = MIX_NEG, l_run = 0.f;                                    // of head tid >> 4 (replicated over its 16 keys' threads)
  bf16x8_t kf[4][DC];
  auto load_k = [&](int t) {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (i < gw && wave * gw + i < p.G) {
        const bf16_t* kr = kb + ((size_t)(wave * gw + i) * p.Tp + t * 16) * p.dimp;
#pragma unroll
        for (int c = 0; c < DC; ++c)
          if (c < dc) kf[i][c] = *(const bf16x8_t*)(kr + c * 32);
      }
  };
  load_k(t_begin);
  for (int t = t_begin; t < t_end; ++t) {
    // ---- value rows of this tile: requested now, used after the softmax
    u32x4_t vv[NP][2];
#pragma unroll
    for (int j = 0; j < NP; ++j) {
      const int i = min(tid + 512 * j, p.H * p.vdim - 1), h = i / p.vdim, d = i - h * p.vdim;
      const u32x4_t* vr = (const u32x4_t*)((const bf16_t*)p.v + ((((size_t)b * p.G + h / per) * (p.Tp >> 4) + t) * p.vdimp + d) * 16);
      vv[j][0] = vr[0], vv[j][1] = vr[1];
    }
    // ---- raw scores: rows = keys, columns = the query heads of a kv head
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (i < gw && wave * gw + i < p.G) {
        const int g = wave * gw + i;
        f32x4_t s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int c = 0; c < DC; ++c)
          if (c < dc) {
            const bf16x8_t qf = *(const bf16x8_t*)(qs + (size_t)(g * per + min(lc, per - 1)) * p.dimp + c * 32 + lg * 8);
            s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[i][c], qf, s, 0, 0, 0);
          }
        if (lc < per) *(float4*)(S + (g * per + lc) * SS + lg * 4) = make_float4(s[0], s[1], s[2], s[3]);
      }
    if (t + 1 < t_end) load_k(t + 1);
    __syncthreads();
    // ---- mixing + softmax: thread = (head, key)
    {
      const int h = tid >> 4, key = t * 16 + lc;
      if (h < p.H) {
        float s = 0.f;
        for (int g = 0; g < p.H; ++g) s = fmaf(talk[h * (MIX_MAX_H + 1) + g], S[g * SS + lc], s);
        s = key <= past && key >= first ? s * sc : -INFINITY;
        const float mn = fmaxf(m_run, row16_max(s)), al = __builtin_amdgcn_exp2f(m_run - mn), e = __builtin_amdgcn_exp2f(s - mn);
        m_run = mn;
        l_run = l_run * al + row16_sum(e);
        P[h * SS + lc] = e;
        if (lc == 0) AL[h] = al;
      }
    }
    __syncthreads();
#pragma unroll
    for (int j = 0; j < NP; ++j) {
      const int i = min(tid + 512 * j, p.H * p.vdim - 1), h = i / p.vdim;
      const float* pr = P + h * SS;
      float a = acc[j] * AL[h];
#pragma unroll
      for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int w = 0; w < 4; ++w) {
          a = fmaf(pr[u * 8 + 2 * w], bf16lo(vv[j][u][w]), a);
          a = fmaf(pr[u * 8 + 2 * w + 1], bf16hi(vv[j][u][w]), a);
        }
      acc[j] = a;
    }
  }
  if (lc == 0 && (tid >> 4) < p.H) *(f32x2_t*)(ml + 2 * (tid >> 4)) = (f32x2_t){m_run, l_run};
  float* od = ws_o(p.ws, p, p.B, b, split);
#pragma unroll
  for (int j = 0; j < NP; ++j)
    if (tid + 512 * j < p.H * p.vdim) od[tid + 512 * j] = acc[j];
}

// ---------------------------------------------------------------- merge of the splits + sink + output gate
__global__ void __launch_bounds__(256) k_attn_mix_combine(AttnMixP p) {
  __shared__ float red[16], part[256];
  const int h = blockIdx.x, tid = threadIdx.x;
  const size_t row = blockIdx.y, rows = (size_t)p.B * p.L;
  int n = p.n_split;
  if (p.tiles_per_split) {                                               // decode: only the runs that reach into the live keys were written
    const int past = p.d_past ? *p.d_past : p.past;
    n = min(n, (past >> 4) / p.tiles_per_split + 1);
  }
  const float sk = bf16_to_f32(p.sink[h]) * LOG2E;
  float m = sk;
  for (int s = tid; s < n; s += 256) m = fmaxf(m, ws_ml(p.ws, p, row, s)[2 * h]);
  m = block_max(m, red);
  float l = 0.f;
  for (int s = tid; s < n; s += 256) { const float* q = ws_ml(p.ws, p, row, s) + 2 * h; l += q[1] * __builtin_amdgcn_exp2f(q[0] - m); }
  l = block_sum(l, red) + __builtin_amdgcn_exp2f(sk - m);
  const float f = gate_of((const bf16_t*)p.gate + row * p.ld + h) / l;
  const int vw = p.vdim <= 32 ? 32 : p.vdim <= 64 ? 64 : p.vdim <= 128 ? 128 : 256, ng = 256 / vw, grp = tid / vw;
  for (int d0 = 0; d0 < p.vdim; d0 += vw) {
    const int d = d0 + tid - grp * vw;
    float a = 0.f;
    if (d < p.vdim)
#pragma unroll 4
      for (int s = grp; s < n; s += ng) {
        const float ms = ws_ml(p.ws, p, row, s)[2 * h];
        if (ms > 0.5f * MIX_NEG) a = fmaf(__builtin_amdgcn_exp2f(ms - m), ws_o(p.ws, p, rows, row, s)[(size_t)h * p.vdim + d], a);
      }
    __syncthreads();
    part[tid] = a;
    __syncthreads();
    if (grp == 0 && d < p.vdim) {
      for (int g = 1; g < ng; ++g) a += part[g * vw + tid];
      ((bf16_t*)p.out)[row * p.H * p.vdim + (size_t)h * p.vdim + d] = f32_to_bf16(a * f);
    }
  }
}

// ---------------------------------------------------------------- host side
static bool mix_fast(int H, int G, int dim, int vdim, int f32) {
  return !f32 && H <= MIX_MAX_H && dim <= 128 && vdim <= 128;
}

extern "C" int p3v_attn_mix_plan(int B, int L, int H, int G, int dim, int vdim, int n_keys, int f32) {
  if (B <= 0 || L <= 0 || H <= 0 || G <= 0 || n_keys <= 0 || !mix_fast(H, G, dim, vdim, f32)) return 0;
  const int want = p3v_tuning().mix_wgs;
  if (L == 1) return max(1, min(p3v_cdiv(n_keys, 16), (want > 0 ? want : 512) / B));
  const int qt = p3v_cdiv(L, 16) * B, tiles = p3v_cdiv(n_keys, 32);
  return max(1, min(min(16, p3v_cdiv(want > 0 ? want : 320, qt)), tiles / 4));
}

extern "C" int64_t p3v_attn_mix_ws_bytes(int B, int L, int H, int vdim, int n_split) {
  if (B <= 0 || L <= 0 || H <= 0 || vdim <= 0 || n_split <= 0) return 0;
  return (int64_t)B * L * n_split * H * (vdim + 2) * 4;
}

static int mix_combine(const AttnMixP& p, hipStream_t s) {
  hipLaunchKernelGGL(k_attn_mix_combine, dim3(p.H, p.B * p.L), dim3(256), 0, s, p);
  P3V_CHECK_LAUNCH();
  return P3V_OK;
}

template <int HW, int DC>
static int launch_prefill(const AttnMixP& p, hipStream_t s) {
  static bool attr_set = false;
  if (!attr_set) {
    if (hipFuncSetAttribute((const void*)k_attn_mix_prefill<HW, DC>, hipFuncAttributeMaxDynamicSharedMemorySize, MixCfg<HW>::LDS) != hipSuccess) return P3V_ERR_HIP;
    attr_set = true;
  }
  hipLaunchKernelGGL((k_attn_mix_prefill<HW, DC>), dim3(p3v_cdiv(p.L, 16), p.n_split, p.B), dim3(512), MixCfg<HW>::LDS, s, p);
  P3V_CHECK_LAUNCH();
  return p.n_split > 1 ? mix_combine(p, s) : P3V_OK;
}
template <int HW>
static int prefill_dc(const AttnMixP& p, hipStream_t s) {
  const int dc = max(p.dimp / 32, p3v_cdiv(p.vdimp, 32));
  switch (dc) {
    case 1: return launch_prefill<HW, 1>(p, s);
    case 2: return launch_prefill<HW, 2>(p, s);
    case 3: return launch_prefill<HW, 3>(p, s);
    default: return launch_prefill<HW, 4>(p, s);
  }
}

extern "C" int p3v_attn_mix(const p3v_mix_args_t* a, void* stream) {
  const int rc = p3v_mix_check(a);
  if (rc != P3V_OK) return rc;
  if (!a->q || !a->talk || !a->sink || !a->gate || !a->out || a->n_split < 0) return P3V_ERR_ARG;
  hipStream_t s = (hipStream_t)stream;
  if (a->n_split == 0 || !mix_fast(a->H, a->G, a->dim, a->vdim, a->f32)) return p3v_attn_mix_any(a, s);
  if (a->n_split > 1 && !a->ws) return P3V_ERR_ARG;
  const AttnMixP p = attn_mix_params(a);
  return p.H <= 8 ? prefill_dc<1>(p, s) : p.H <= 16 ? prefill_dc<2>(p, s) : prefill_dc<4>(p, s);
}

template <int DC, int NP>
static int launch_decode(const QkvHeadsP& hp, const AttnMixP& p, hipStream_t s) {
  hipLaunchKernelGGL((k_attn_mix_decode<DC, NP>), dim3(p.n_split, p.B), dim3(512), (size_t)p.H * p.dimp * 2, s, hp, p);
  P3V_CHECK_LAUNCH();
  return mix_combine(p, s);
}
template <int DC>
static int decode_np(const QkvHeadsP& hp, const AttnMixP& p, hipStream_t s) {
  const int np = p3v_cdiv(p.H * p.vdim, 512);
  return np <= 1 ? launch_decode<DC, 1>(hp, p, s) : np <= 2 ? launch_decode<DC, 2>(hp, p, s) : np <= 4 ? launch_decode<DC, 4>(hp, p, s)
       : np <= 6 ? launch_decode<DC, 6>(hp, p, s) : launch_decode<DC, 8>(hp, p, s);
}

extern "C" int p3v_attn_mix_decode(const p3v_mix_args_t* a, void* stream) {
  const int rc = p3v_mix_check(a);
  if (rc != P3V_OK) return rc;
  if (!a->qkv || !a->q_norm || !a->k_norm || !a->talk || !a->sink || !a->gate || !a->out || a->n_split < 0) return P3V_ERR_ARG;
  if (a->L != 1 || a->n_split == 0 || !mix_fast(a->H, a->G, a->dim, a->vdim, a->f32) || a->H / a->G > 16) return P3V_ERR_UNSUPPORTED;
  if (!a->ws) return P3V_ERR_ARG;
  AttnMixP p = attn_mix_params(a);
  p.tiles_per_split = p3v_cdiv(a->Tp / 16, a->n_split);
  const QkvHeadsP hp = {a->qkv, a->q_norm, a->k_norm, a->v_first, nullptr, a->k, a->v, a->d_past, a->eps, a->vmix,
                        a->B, a->L, a->H, a->G, a->dim, a->vdim, a->dimp, a->vdimp, a->ld, a->ld_first, a->past, a->Tp};
  hipStream_t s = (hipStream_t)stream;
  switch (a->dimp / 32) {
    case 1: return decode_np<1>(hp, p, s);
    case 2: return decode_np<2>(hp, p, s);
    case 3: return decode_np<3>(hp, p, s);
    default: return decode_np<4>(hp, p, s);
  }
}
