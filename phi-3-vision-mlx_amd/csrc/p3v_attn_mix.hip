// Attention whose heads' scores are mixed before the softmax (score_h <- sum_g talk[h, g] score_g), with a per-head sink in the
// denominator and a per-head output gate.  The mixing couples ALL heads at every (query, key) pair, so a workgroup owns all heads of
// its queries (one head per workgroup, the usual split, would recompute every head's scores in every workgroup).
//
//   K cache [B, G, Tp, dimp]            rows of keys: a row is an MFMA fragment (dimp: dim rounded up to 32, zeros behind)
//   V cache [B, G, Tp / 16, vdimp, 16]  blocks of 16 keys, value dimension by value dimension: the PV product reads 8 consecutive
//                                       keys of one dimension per lane (16 bytes, whole 512-byte runs per wave) and a 16-key tile of
//                                       the decode step is contiguous (vdimp: vdim rounded up to 32)
//
// Scores, their mixing and the softmax are fp32.  The mixing runs on the bf16 matrix cores WITHOUT losing fp32: talk is bf16 data, and
// a score is split into three bf16 terms whose sum is the fp32 value, so that every product is exact and only the fp32 accumulation
// rounds -- an eighth of the cost of the fp32 matrix instruction.
#include "p3v_layered.h"

#define MIX_NEG (-1e30f)             // "no key yet": finite, so that differences of two of them stay 0
#define MIX_MAX_H 32
#define LOG2E 1.4426950408889634f

typedef __attribute__((ext_vector_type(2))) float f32x2_t;

// workgroup barrier for LDS data only: global loads stay in flight across it (__syncthreads would wait for them)
__device__ __forceinline__ void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}
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
//   P  [heads][16 q][32 keys] bf16,  AL [heads][16 q] rescale factors,  MM [heads][16 q] running maxima
// The softmax's sum rides in the second product as one more value dimension (a row of ones).  The value fragments of a tile are
// requested ahead of its mixing and the next tile's key fragments ahead of the second product; the barriers wait for LDS only.
// SHARED: the heads of a wave share one key / value head (else every head loads its own fragments, one head ahead).
template <int HW> struct MixCfg {
  static constexpr int HP = 8 * HW, HS = HP + 4, QS = 32 * HS + 4;      // heads padded, S strides (floats): key, query
  static constexpr int PQ = 40, PH = 16 * PQ + 8;                        // P strides (bf16): query, head
  static constexpr int HM = (HP + 15) / 16;                              // 16-head row blocks of the mixing
  static constexpr int S_BYTES = 16 * QS * 4, P_BYTES = HP * PH * 2, A_BYTES = HM * 16 * 16 * 4;
  static constexpr int LDS = S_BYTES + P_BYTES + 2 * A_BYTES + HM * 1024 + (HW == 4 ? 8 * 4096 : 0);
};

template <int HW, int DC, int VC, bool SHARED>
__global__ void __launch_bounds__(512, 1) k_attn_mix_prefill(AttnMixP p) {
  typedef MixCfg<HW> C;
  constexpr int NB = SHARED ? 1 : 2;                                     // fragment buffers
  constexpr int QU = HW == 4 && DC + VC >= 5 ? 1 : 2;                    // queries of the mixing side by side
  constexpr bool Q_REG = HW < 4 || DC + VC <= 6;                         // else the query fragments are read again for every key tile
  constexpr bool Q_LDS = HW == 4 && DC + VC == 6;                        // the last head's wait in LDS
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  float* S = (float*)smem;
  bf16_t* P = (bf16_t*)(smem + C::S_BYTES);
  float* AL = (float*)(smem + C::S_BYTES + C::P_BYTES);
  float* MM = AL + C::HM * 256;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lc = lane & 15, lg = lane >> 4;
  const int n_qt = (p.L + 15) >> 4, qt = n_qt - 1 - (int)blockIdx.x, split = blockIdx.y, b = blockIdx.z;   // longest rows first
  const int q0 = qt * 16, per = p.H / p.G, past = p.d_past ? *p.d_past : p.past, first = p.pad_len ? p.pad_len[b] : 0;
  const int last = past + min(q0 + 15, p.L - 1);                         // last key any query of the tile sees
  // key tiles of this split: the same for every query tile, so that the workgroups an XCD runs together walk the same keys (its L2
  // then serves all but the first); splits beyond a query tile's keys have nothing to do and nobody reads their partials
  const int t0 = max(first >> 5, split * p.tiles_per_split), t1 = min((last >> 5) + 1, (split + 1) * p.tiles_per_split);
  if (split * p.tiles_per_split > last >> 5) return;
  constexpr int NV = 2 * VC;                                             // 16-dimension blocks of a value (dimp = 32 DC, vdimp = 32 VC)
  const float sc = fabsf(p.scale) * LOG2E;                               // (a negative scale's sign goes into talk: the row maxima then scale)
  const uint32_t flip = p.scale < 0.f ? 0x8000u : 0u;

  // Q fragments (B operand: column = query, 8 consecutive dimensions)
  u32x4_t* QL = (u32x4_t*)(MM + C::HM * 256) + C::HM * 64 + wave * (4 * 64) + lane;
  bf16x8_t qf[Q_REG ? HW : 1][DC];
  auto load_q = [&](int i) {
    const int h = min(wave * HW + i, p.H - 1);
    const bf16_t* qr = (const bf16_t*)p.q + (((size_t)b * p.H + h) * p.L + min(q0 + lc, p.L - 1)) * p.dimp + lg * 8;
#pragma unroll
    for (int c = 0; c < DC; ++c) {
      const bf16x8_t v = *(const bf16x8_t*)(qr + c * 32);
      if (Q_LDS && i == HW - 1) QL[c * 64] = __builtin_bit_cast(u32x4_t, v);
      else qf[Q_REG ? i : 0][c] = v;
    }
  };
  if constexpr (Q_REG) {
#pragma unroll
    for (int i = 0; i < HW; ++i) load_q(i);
  }
  // talk fragments (A operand: row = mixed head, 8 consecutive raw heads), zero beyond H; kept in LDS
  u32x4_t* TF = (u32x4_t*)(MM + C::HM * 256);
  for (int m = wave; m < C::HM; m += 8) {
    u32x4_t w = {0u, 0u, 0u, 0u};
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int h = m * 16 + lc, g = lg * 8 + j;
      const uint32_t v = h < p.H && g < p.H ? p.talk[h * p.H + g] ^ flip : 0;
      w[j >> 1] |= v << (16 * (j & 1));
    }
    TF[m * 64 + lane] = w;
  }
  f32x4_t o[HW][NV], ol = {0.f, 0.f, 0.f, 0.f};                          // outputs; softmax sums (row i: head i of the wave)
#pragma unroll
  for (int i = 0; i < HW; ++i) {
#pragma unroll
    for (int d = 0; d < NV; ++d) o[i][d] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
  }
  for (int i = tid; i < C::HM * 256; i += 512) MM[i] = MIX_NEG;
  if (p.H < C::HP)                                                       // heads that no wave writes: finite, talk's zero columns do the rest
    for (int i = tid; i < C::S_BYTES / 4; i += 512) S[i] = 0.f;
  lds_barrier();

  const bf16_t* kb = (const bf16_t*)p.k + (size_t)b * p.G * p.Tp * p.dimp;
  const bf16_t* vb = (const bf16_t*)p.v + (size_t)b * p.G * p.Tp * p.vdimp;
  const uint32_t k_lane = (uint32_t)(lc * p.dimp + lg * 8), v_lane = (uint32_t)(((lg >> 1) * p.vdimp + lc) * 16 + (lg & 1) * 8);
  const bool active = wave * HW < p.H;
  bf16x8_t kf[NB][2][DC], vf[NB][NV];
  auto load_k = [&](int t, int i) {
    const int g = min(wave * HW + i, p.H - 1) / per, bf = SHARED ? 0 : i & 1;
    const bf16_t *k0 = kb + ((size_t)g * p.Tp + t * 32) * p.dimp, *k1 = k0 + (size_t)16 * p.dimp;
    asm volatile("" : "+s"(k0), "+s"(k1));                               // (scalar bases + one 32-bit lane offset: no 64-bit lane addresses)
#pragma unroll
    for (int c = 0; c < DC; ++c) kf[bf][0][c] = *(const bf16x8_t*)(k0 + k_lane + c * 32), kf[bf][1][c] = *(const bf16x8_t*)(k1 + k_lane + c * 32);
  };
  auto load_v = [&](int t, int i) {
    const int g = min(wave * HW + i, p.H - 1) / per, bf = SHARED ? 0 : i & 1;
    const bf16_t* vr = vb + ((size_t)g * (p.Tp >> 4) + t * 2) * p.vdimp * 16;
    asm volatile("" : "+s"(vr));
#pragma unroll
    for (int d = 0; d < NV; ++d)
      vf[bf][d] = *(const bf16x8_t*)(vr + v_lane + d * 256);
  };
  if (active && t0 < t1) load_k(t0, 0);

  for (int t = t0; t < t1; ++t) {
    // ---- raw scores of this wave's heads -> S
    if (active) {
      f32x4_t s[HW][2];
#pragma unroll
      for (int i = 0; i < HW; ++i) {
        s[i][0] = s[i][1] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
        if (!SHARED && i + 1 < HW) load_k(t, i + 1);
        if constexpr (!Q_REG) load_q(i);
#pragma unroll
        for (int c = 0; c < DC; ++c)
          {
            bf16x8_t q;
            if (Q_LDS && i == HW - 1) q = __builtin_bit_cast(bf16x8_t, QL[c * 64]);
            else q = qf[Q_REG ? i : 0][c];
            s[i][0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[SHARED ? 0 : i & 1][0][c], q, s[i][0], 0, 0, 0);
            s[i][1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[SHARED ? 0 : i & 1][1][c], q, s[i][1], 0, 0, 0);
          }
        if (HW > 1) __builtin_amdgcn_sched_barrier(0);
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
      load_v(t, 0);
    }
    lds_barrier();

    // ---- mixing + softmax of queries 2w, 2w + 1, all heads; a lane's two keys are neighbours (2 lc, 2 lc + 1)
    const bool edge = t * 32 + 31 > past + q0 || t * 32 < first;         // some query of the tile does not see some key
#pragma unroll QU
    for (int qi = 0; qi < 2; ++qi) {
      const int q = 2 * wave + qi;
      f32x4_t mx[C::HM][2];
      float mo[C::HM][4];
#pragma unroll
      for (int m = 0; m < C::HM; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) mo[m][r] = MM[(m * 16 + lg * 4 + r) * 16 + q];
#pragma unroll
      for (int kt = 0; kt < 2; ++kt) {
        float v[8];
        const float* src = S + q * C::QS + (2 * lc + kt) * C::HS + lg * 8;
        if (C::HP == 32 || lg * 8 < C::HP) {
          const float4 a = *(const float4*)src, c = *(const float4*)(src + 4);
          v[0] = a.x, v[1] = a.y, v[2] = a.z, v[3] = a.w, v[4] = c.x, v[5] = c.y, v[6] = c.z, v[7] = c.w;
        } else {
#pragma unroll
          for (int j = 0; j < 8; ++j) v[j] = 0.f;
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
          const bf16x8_t tf = __builtin_bit_cast(bf16x8_t, TF[m * 64 + lane]);
#pragma unroll
          for (int k = 2; k >= 0; --k) a = __builtin_amdgcn_mfma_f32_16x16x32_bf16(tf, __builtin_bit_cast(bf16x8_t, part[k]), a, 0, 0, 0);
          mx[m][kt] = a;
        }
      }
      if (edge) {
        const int qpos = past + q0 + q, key0 = t * 32 + 2 * lc;
        const bool live0 = key0 <= qpos && key0 >= first, live1 = key0 < qpos && key0 + 1 >= first;
#pragma unroll
        for (int m = 0; m < C::HM; ++m)
#pragma unroll
          for (int r = 0; r < 4; ++r) mx[m][0][r] = live0 ? mx[m][0][r] : -INFINITY, mx[m][1][r] = live1 ? mx[m][1][r] : -INFINITY;
      }
      float rm[C::HM * 4];                                               // row maxima over the 16 lanes: stage by stage, so that no lane move waits
#pragma unroll
      for (int i = 0; i < C::HM * 4; ++i) rm[i] = fmaxf(mx[i >> 2][0][i & 3], mx[i >> 2][1][i & 3]);
#define MIX_ROWS_STAGE(ctrl)                                                                              \
  _Pragma("unroll") for (int i = 0; i < C::HM * 4; ++i) rm[i] = fmaxf(rm[i], P3V_DPP_F32(rm[i], ctrl));   \
  __builtin_amdgcn_sched_barrier(0);
      MIX_ROWS_STAGE(0xB1) MIX_ROWS_STAGE(0x4E) MIX_ROWS_STAGE(0x124) MIX_ROWS_STAGE(0x128)
#undef MIX_ROWS_STAGE
      float al_k = 0.f, mn_k = 0.f;                                      // of row (lc >> 2, lc & 3): what this lane writes
#pragma unroll
      for (int m = 0; m < C::HM; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float mn = fmaxf(mo[m][r], rm[m * 4 + r] * sc), al = __builtin_amdgcn_exp2f(mo[m][r] - mn);
          const float p0 = __builtin_amdgcn_exp2f(fmaf(mx[m][0][r], sc, -mn)), p1 = __builtin_amdgcn_exp2f(fmaf(mx[m][1][r], sc, -mn));
          if (C::HP >= 16 || lg < 2) *(uint32_t*)(P + (m * 16 + lg * 4 + r) * C::PH + q * C::PQ + 2 * lc) = pack_bf16x2(p0, p1);
          al_k = lc == m * 4 + r ? al : al_k, mn_k = lc == m * 4 + r ? mn : mn_k;
        }
      if (lc < 4 * C::HM && (C::HP >= 16 || lg < 2)) {
        const int h = (lc >> 2) * 16 + lg * 4 + (lc & 3);
        AL[h * 16 + q] = al_k, MM[h * 16 + q] = mn_k;
      }
    }
    lds_barrier();

    // ---- O^T += V^T P^T of this wave's heads
    if (active) {
      load_k(min(t + 1, t1 - 1), 0);
#pragma unroll
      for (int i = 0; i < HW; ++i) {
        const int h = min(wave * HW + i, p.H - 1);
        if (!SHARED && i + 1 < HW) load_v(t, i + 1);
        const bf16x8_t pf = *(const bf16x8_t*)(P + h * C::PH + lc * C::PQ + lg * 8);
        const float al = AL[h * 16 + lc];
        if (__builtin_amdgcn_ballot_w64(al != 1.f)) {                    // (a maximum moved; rare behind a sequence's first tiles)
          ol[i] *= lg == 0 ? al : 1.f;
#pragma unroll
          for (int d = 0; d < NV; ++d) o[i][d] *= al;
        }
        uint32_t one = lc == i ? 0x3f803f80u : 0u;                       // A: a row of ones at row i
        asm volatile("" : "+v"(one));                                    // (not kept in registers across the loop, one fragment per head)
        const u32x4_t ones = {one, one, one, one};
        ol = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, ones), pf, ol, 0, 0, 0);
#pragma unroll
        for (int d = 0; d < NV; ++d)
          o[i][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[SHARED ? 0 : i & 1][d], pf, o[i][d], 0, 0, 0);
        if (HW > 1) __builtin_amdgcn_sched_barrier(0);                   // (one head's operands at a time: the registers are full)
      }
    }
  }

  const int row_q = q0 + lc;
  if (!active || row_q >= p.L) return;
  const size_t row = (size_t)b * p.L + row_q, rows = (size_t)p.B * p.L;
#pragma unroll
  for (int i = 0; i < HW; ++i) {
    const int h = wave * HW + i;
    if (h >= p.H) continue;
    const float m = MM[h * 16 + lc], l = __shfl(ol[i], lc, 64);           // (the sums sit in the first 16 lanes)
    float f = 1.f;
    if (p.n_split == 1) {
      const float sk = bf16_to_f32(p.sink[h]) * LOG2E, mm = fmaxf(m, sk), e = __builtin_amdgcn_exp2f(m - mm);
      f = e / (l * e + __builtin_amdgcn_exp2f(sk - mm)) * gate_of((const bf16_t*)p.gate + row * p.ld + h);
    } else if (lg == 0) {
      *(f32x2_t*)(ws_ml(p.ws, p, row, split) + h * 2) = (f32x2_t){m, l};
    }
#pragma unroll
    for (int d = 0; d < NV; ++d)
      {
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
          if (p.vdim % 4 == 0) {
            if (dd < p.vdim) *(float4*)dst = make_float4(o[i][d][0], o[i][d][1], o[i][d][2], o[i][d][3]);
          } else {
#pragma unroll
            for (int r = 0; r < 4; ++r)
              if (dd + r < p.vdim) dst[r] = o[i][d][r];
          }
        }
      }
  }
}

// ================================================================ one new token per sequence
// A workgroup takes a run of 16-key tiles of one sequence, all heads: the query's whole-projection norm is recomputed in every
// workgroup (a few KB), the workgroup whose run holds the new position also normalises and appends the new key and mixes and appends
// the new value.  Partials of the runs are merged by k_attn_mix_combine.
template <int GW, int DC, int NP, bool VEC>
__global__ void __launch_bounds__(512) k_attn_mix_decode(QkvHeadsP hp, AttnMixP p) {
  constexpr int SS = 20;                                                 // S / P row stride (floats)
  __shared__ float S[MIX_MAX_H * SS], P[MIX_MAX_H * SS], talk[MIX_MAX_H * (MIX_MAX_H + 1)], AL[MIX_MAX_H], red[2][8];
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  bf16_t* qs = (bf16_t*)smem;                                            // [H][dimp] normalised query
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lc = lane & 15, lg = lane >> 4;
  const int split = blockIdx.x, b = blockIdx.y, per = p.H / p.G;
  const int past = p.d_past ? *p.d_past : p.past, first = p.pad_len ? p.pad_len[b] : 0;
  const int t_first = split * p.tiles_per_split, own = past >> 4;
  if (t_first > own) return;                                             // beyond the live keys: the merge does not look here
  const int t_begin = max(t_first, first >> 4), t_end = min(t_first + p.tiles_per_split, own + 1);
  const bool owner = own < t_first + p.tiles_per_split;
  const int nq = p.H * p.dim, nk = p.G * p.dim, nv = p.G * p.vdim;
  const bf16_t* row = (const bf16_t*)hp.qkv + (size_t)b * hp.ld;
  float* ml = ws_ml(p.ws, p, b, split);
  if (t_begin >= t_end) {                                                // only padding here (and the new position is in no such run)
    for (int h = tid; h < p.H; h += 512) ml[2 * h] = MIX_NEG, ml[2 * h + 1] = 0.f;
    if (!owner) return;                                                  // an idle batch row still appends: its cache stays finite
  }

  // ---- keys and values of the first tile are requested before anything else (by the workgroup of the new position behind its append)
  // (GW kv heads per wave; a wave beyond the last one repeats it: same loads, same scores)
  const float sc = p.scale * LOG2E;
  const bf16_t* kb = (const bf16_t*)p.k + ((size_t)b * p.G * p.Tp + lc) * p.dimp + lg * 8;
  bf16x8_t kf[GW][DC];
  auto load_k = [&](int t) {
#pragma unroll
    for (int i = 0; i < GW; ++i) {
      const bf16_t* kr = kb + ((size_t)min(wave * GW + i, p.G - 1) * p.Tp + t * 16) * p.dimp;
#pragma unroll
      for (int c = 0; c < DC; ++c) kf[i][c] = *(const bf16x8_t*)(kr + c * 32);
    }
  };
  u32x4_t vv[NP][2];
  int vh[NP];
  uint32_t vo[NP];
#pragma unroll
  for (int j = 0; j < NP; ++j) {
    const int i = min(tid + 512 * j, p.H * p.vdim - 1), h = i / p.vdim, d = i - h * p.vdim, g = h / per;
    vh[j] = h;
    vo[j] = (uint32_t)(g * (p.Tp >> 4) * p.vdimp + d) * 2;               // 16-byte units inside the sequence's cache
  }
  const u32x4_t* vb = (const u32x4_t*)p.v + (size_t)b * p.G * (p.Tp >> 4) * p.vdimp * 2;
  auto load_v = [&](int t) {
#pragma unroll
    for (int j = 0; j < NP; ++j) {
      const u32x4_t* vr = vb + vo[j] + (uint32_t)t * (uint32_t)(p.vdimp * 2);
      vv[j][0] = vr[0], vv[j][1] = vr[1];
    }
  };
  // ---- query (and key) norm.  VEC: 8 columns per thread, read once, together with the weights
  constexpr u32x4_t zero4 = {0u, 0u, 0u, 0u};
  u32x4_t qv = zero4, qw = zero4, kv = zero4, kw = zero4, nw = zero4, fw = zero4;
  const int e8 = tid * 8;
  float sq = 0.f, sk = 0.f;
  if constexpr (VEC) {
    if (e8 < nq) qv = *(const u32x4_t*)(row + e8), qw = *(const u32x4_t*)(hp.q_norm + e8);
    if (owner) {
      if (e8 < nk) kv = *(const u32x4_t*)(row + nq + e8), kw = *(const u32x4_t*)(hp.k_norm + e8);
      if (e8 < nv) {
        nw = *(const u32x4_t*)(row + nq + nk + e8);
        if (hp.v_first) fw = *(const u32x4_t*)((const bf16_t*)hp.v_first + (size_t)b * hp.ld_first + e8);
      }
    }
    if (!owner) load_k(t_begin), load_v(t_begin);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      sq += bf16lo(qv[j]) * bf16lo(qv[j]) + bf16hi(qv[j]) * bf16hi(qv[j]);
      sk += bf16lo(kv[j]) * bf16lo(kv[j]) + bf16hi(kv[j]) * bf16hi(kv[j]);
    }
  } else {
    for (int e = tid; e < nq; e += 512) { const float v = bf16_to_f32(row[e]); sq += v * v; }
    if (owner)
      for (int e = tid; e < nk; e += 512) { const float v = bf16_to_f32(row[nq + e]); sk += v * v; }
    if (!owner) load_k(t_begin), load_v(t_begin);
  }
  for (int e = tid; e < p.H * p.H; e += 512) { const int h = e / p.H; talk[h * (MIX_MAX_H + 1) + e - h * p.H] = bf16_to_f32(p.talk[e]); }
  sq = wave_sum(sq), sk = wave_sum(sk);
  if (lane == 0) red[0][wave] = sq, red[1][wave] = sk;
  lds_barrier();                                                         // (the tile's loads stay in flight)
  sq = sk = 0.f;
#pragma unroll
  for (int w = 0; w < 8; ++w) sq += red[0][w], sk += red[1][w];
  const float rq = 1.f / sqrtf(sq / (float)nq + hp.eps), rk = 1.f / sqrtf(sk / (float)nk + hp.eps);
  if constexpr (VEC) {
    auto normed = [](u32x4_t x, u32x4_t w, float r) {
      u32x4_t y;
#pragma unroll
      for (int j = 0; j < 4; ++j) y[j] = pack_bf16x2(bf16lo(x[j]) * r * bf16lo(w[j]), bf16hi(x[j]) * r * bf16hi(w[j]));
      return y;
    };
    if (e8 < nq) { const int h = e8 / p.dim; *(u32x4_t*)(qs + h * p.dimp + e8 - h * p.dim) = normed(qv, qw, rq); }
    if (p.dimp != p.dim)
      for (int e = tid; e < p.H * (p.dimp - p.dim); e += 512) { const int h = e / (p.dimp - p.dim); qs[h * p.dimp + p.dim + e - h * (p.dimp - p.dim)] = 0; }
    if (owner) {
      if (e8 < nk) {
        const int g = e8 / p.dim;
        *(u32x4_t*)((bf16_t*)hp.k + (((size_t)b * p.G + g) * p.Tp + past) * p.dimp + e8 - g * p.dim) = normed(kv, kw, rk);
      }
      if (e8 < nv) {
        const int g = e8 / p.vdim;
        bf16_t* dst = (bf16_t*)hp.v + ((((size_t)b * p.G + g) * (p.Tp >> 4) + own) * p.vdimp + e8 - g * p.vdim) * 16 + (past & 15);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          float lo = bf16lo(nw[j]), hi = bf16hi(nw[j]);
          if (hp.v_first) lo = (1.f - hp.vmix) * lo + hp.vmix * bf16lo(fw[j]), hi = (1.f - hp.vmix) * hi + hp.vmix * bf16hi(fw[j]);
          dst[32 * j] = f32_to_bf16(lo), dst[32 * j + 16] = f32_to_bf16(hi);
        }
      }
      __syncthreads();                                                   // (the stores have to be visible to the whole workgroup)
    }
  } else {
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
      __syncthreads();                                                   // (as above)
    }
  }
  lds_barrier();                     // the query (and the new key / value) is in LDS
  if (t_begin >= t_end) return;
  if (owner) load_k(t_begin), load_v(t_begin);

  float acc[NP];
#pragma unroll
  for (int j = 0; j < NP; ++j) acc[j] = 0.f;
  float m_run = MIX_NEG, l_run = 0.f;                                    // of head tid >> 4 (replicated over its 16 keys' threads)
  for (int t = t_begin; t < t_end; ++t) {
    // ---- raw scores: rows = keys, columns = the query heads of a kv head
#pragma unroll
    for (int i = 0; i < GW; ++i) {
      const int g = min(wave * GW + i, p.G - 1);
      f32x4_t s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int c = 0; c < DC; ++c) {
        const bf16x8_t qf = *(const bf16x8_t*)(qs + (size_t)(g * per + min(lc, per - 1)) * p.dimp + c * 32 + lg * 8);
        s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[i][c], qf, s, 0, 0, 0);
      }
      if (lc < per) *(float4*)(S + (g * per + lc) * SS + lg * 4) = make_float4(s[0], s[1], s[2], s[3]);
    }
    if (t + 1 < t_end) load_k(t + 1);
    lds_barrier();
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
    lds_barrier();
#pragma unroll
    for (int j = 0; j < NP; ++j) {
      const float4* pr = (const float4*)(P + vh[j] * SS);
      float a = acc[j] * AL[vh[j]];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const float4 q = pr[u];
        const uint32_t w0 = vv[j][u >> 1][(u & 1) * 2], w1 = vv[j][u >> 1][(u & 1) * 2 + 1];
        a = fmaf(q.x, bf16lo(w0), a), a = fmaf(q.y, bf16hi(w0), a), a = fmaf(q.z, bf16lo(w1), a), a = fmaf(q.w, bf16hi(w1), a);
      }
      asm volatile("" : "+v"(a));                                        // (here, not sunk behind the branch below with every operand kept)
      acc[j] = a;
    }
    if (t + 1 < t_end) load_v(t + 1);
  }
  if (lc == 0 && (tid >> 4) < p.H) *(f32x2_t*)(ml + 2 * (tid >> 4)) = (f32x2_t){m_run, l_run};
  float* od = ws_o(p.ws, p, p.B, b, split);
#pragma unroll
  for (int j = 0; j < NP; ++j)
    if (tid + 512 * j < p.H * p.vdim) od[tid + 512 * j] = acc[j];
}

// ---------------------------------------------------------------- merge of the splits + sink + output gate
// splits of `row` that were written: those that begin at or before its last live key tile
__device__ __forceinline__ int live_splits(const AttnMixP& p, size_t row, int shift) {
  const int past = p.d_past ? *p.d_past : p.past, l = (int)(row % p.L), last = past + min((l & ~15) + 15, p.L - 1);
  return min(p.n_split, (last >> shift) / p.tiles_per_split + 1);
}
// one token per sequence: many splits, few rows -- a workgroup per (head, row), groups of threads share the splits
#define MIX_MAX_SPLIT 1024
__global__ void __launch_bounds__(1024) k_attn_mix_combine(AttnMixP p) {
  constexpr int U = 16;                                                  // splits per thread group whose outputs are requested up front
  __shared__ float red[16], part[1024], wt[MIX_MAX_SPLIT];
  const int h = blockIdx.x, tid = threadIdx.x;
  const size_t row = blockIdx.y, rows = (size_t)p.B * p.L;
  const int n = live_splits(p, row, 4);
  const int vw = p.vdim <= 32 ? 32 : p.vdim <= 64 ? 64 : 128, ng = 1024 / vw, grp = tid / vw, d = tid - grp * vw;
  const float* o = ws_o(p.ws, p, rows, row, 0) + (size_t)h * p.vdim + min(d, p.vdim - 1);
  const size_t step = (size_t)p.H * p.vdim;
  f32x2_t q = {MIX_NEG, 0.f};
  if (tid < n) q = *(const f32x2_t*)(ws_ml(p.ws, p, row, tid) + 2 * h);
  float v[U];
#pragma unroll
  for (int u = 0; u < U; ++u) v[u] = o[min(grp + u * ng, n - 1) * step];
  const float sk = bf16_to_f32(p.sink[h]) * LOG2E, gate = gate_of((const bf16_t*)p.gate + row * p.ld + h);
  const float m = block_max(fmaxf(sk, q[0]), red), w = __builtin_amdgcn_exp2f(q[0] - m);
  wt[tid] = q[0] > 0.5f * MIX_NEG ? w : -1.f;                            // (-1: no such split, or one of padding whose outputs were not written)
  const float f = gate / (block_sum(q[1] * w, red) + __builtin_amdgcn_exp2f(sk - m));
  float a = 0.f;
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int s = grp + u * ng;
    const float x = wt[min(s, MIX_MAX_SPLIT - 1)];
    a = s < n && x >= 0.f ? fmaf(x, v[u], a) : a;
  }
  for (int s = grp + U * ng; s < n; s += ng) a = wt[s] >= 0.f ? fmaf(wt[s], o[s * step], a) : a;
  part[tid] = a;
  __syncthreads();
  if (grp == 0 && d < p.vdim) {
    for (int g = 1; g < ng; ++g) a += part[g * vw + tid];
    ((bf16_t*)p.out)[row * p.H * p.vdim + (size_t)h * p.vdim + d] = f32_to_bf16(a * f);
  }
}
// prompts: few splits, many rows -- a workgroup per row
#define MIX_MAX_ROW_SPLIT 16
__global__ void __launch_bounds__(256) k_attn_mix_combine_rows(AttnMixP p) {
  __shared__ float wt[MIX_MAX_H][MIX_MAX_ROW_SPLIT];
  const size_t row = blockIdx.x, rows = (size_t)p.B * p.L;
  const int tid = threadIdx.x, n = live_splits(p, row, 5);
  if (tid < p.H) {
    const float sk = bf16_to_f32(p.sink[tid]) * LOG2E;
    float m = sk;
    for (int s = 0; s < n; ++s) m = fmaxf(m, ws_ml(p.ws, p, row, s)[2 * tid]);
    float l = __builtin_amdgcn_exp2f(sk - m);
    for (int s = 0; s < n; ++s) {
      const float* q = ws_ml(p.ws, p, row, s) + 2 * tid;
      l += q[1] * __builtin_amdgcn_exp2f(q[0] - m);
    }
    const float f = gate_of((const bf16_t*)p.gate + row * p.ld + tid) / l;
    for (int s = 0; s < n; ++s) wt[tid][s] = f * __builtin_amdgcn_exp2f(ws_ml(p.ws, p, row, s)[2 * tid] - m);
  }
  __syncthreads();
  const size_t step = (size_t)p.H * p.vdim;
  const float* o = ws_o(p.ws, p, rows, row, 0);
  bf16_t* out = (bf16_t*)p.out + row * step;
  if (p.vdim % 4 == 0) {
    for (int e = tid * 4; e < p.H * p.vdim; e += 1024) {
      const int h = e / p.vdim;
      float4 a = make_float4(0.f, 0.f, 0.f, 0.f);
      for (int s = 0; s < n; ++s) {
        const float4 v = *(const float4*)(o + s * step + e);
        const float w = wt[h][s];
        a.x = fmaf(w, v.x, a.x), a.y = fmaf(w, v.y, a.y), a.z = fmaf(w, v.z, a.z), a.w = fmaf(w, v.w, a.w);
      }
      *(u32x2_t*)(out + e) = (u32x2_t){pack_bf16x2(a.x, a.y), pack_bf16x2(a.z, a.w)};
    }
  } else {
    for (int e = tid; e < p.H * p.vdim; e += 256) {
      float a = 0.f;
      for (int s = 0; s < n; ++s) a = fmaf(wt[e / p.vdim][s], o[s * step + e], a);
      out[e] = f32_to_bf16(a);
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
  if (L == 1) {                                                          // about one workgroup per CU, runs of equal length
    const int tiles = p3v_cdiv(n_keys, 16), per = p3v_cdiv(tiles, max(1, (want > 0 ? want : 256) / B));
    return min(p3v_cdiv(tiles, per), MIX_MAX_SPLIT);
  }
  const int qt = p3v_cdiv(L, 16) * B, tiles = p3v_cdiv(n_keys, 32);
  return max(1, min(min(MIX_MAX_ROW_SPLIT, p3v_cdiv(want > 0 ? want : 320, qt)), tiles / 4));
}

extern "C" int64_t p3v_attn_mix_ws_bytes(int B, int L, int H, int vdim, int n_split) {
  if (B <= 0 || L <= 0 || H <= 0 || vdim <= 0 || n_split <= 0) return 0;
  return (int64_t)B * L * n_split * H * (vdim + 2) * 4;
}

static int mix_combine(const AttnMixP& p, hipStream_t s) {
  if (p.L == 1) hipLaunchKernelGGL(k_attn_mix_combine, dim3(p.H, p.B), dim3(1024), 0, s, p);
  else hipLaunchKernelGGL(k_attn_mix_combine_rows, dim3(p.B * p.L), dim3(256), 0, s, p);
  P3V_CHECK_LAUNCH();
  return P3V_OK;
}

template <int HW, int DC, int VC, bool SHARED>
static int launch_prefill(const AttnMixP& p, hipStream_t s) {
  static bool attr_set = false;
  if (!attr_set) {
    if (hipFuncSetAttribute((const void*)k_attn_mix_prefill<HW, DC, VC, SHARED>, hipFuncAttributeMaxDynamicSharedMemorySize, MixCfg<HW>::LDS) != hipSuccess) return P3V_ERR_HIP;
    attr_set = true;
  }
  hipLaunchKernelGGL((k_attn_mix_prefill<HW, DC, VC, SHARED>), dim3(p3v_cdiv(p.L, 16), p.n_split, p.B), dim3(512), MixCfg<HW>::LDS, s, p);
  P3V_CHECK_LAUNCH();
  return p.n_split > 1 ? mix_combine(p, s) : P3V_OK;
}
template <int HW, bool SHARED, int DC>
static int prefill_vc(const AttnMixP& p, hipStream_t s) {
  switch (p.vdimp / 32) {
    case 1: return launch_prefill<HW, DC, 1, SHARED>(p, s);
    case 2: return launch_prefill<HW, DC, 2, SHARED>(p, s);
    case 3: return launch_prefill<HW, DC, 3, SHARED>(p, s);
    default: return launch_prefill<HW, DC, 4, SHARED>(p, s);
  }
}
template <int HW, bool SHARED>
static int prefill_dc(const AttnMixP& p, hipStream_t s) {
  switch (p.dimp / 32) {
    case 1: return prefill_vc<HW, SHARED, 1>(p, s);
    case 2: return prefill_vc<HW, SHARED, 2>(p, s);
    case 3: return prefill_vc<HW, SHARED, 3>(p, s);
    default: return prefill_vc<HW, SHARED, 4>(p, s);
  }
}

extern "C" int p3v_attn_mix(const p3v_mix_args_t* a, void* stream) {
  const int rc = p3v_mix_check(a);
  if (rc != P3V_OK) return rc;
  if (!a->q || !a->talk || !a->sink || !a->gate || !a->out || a->n_split < 0) return P3V_ERR_ARG;
  hipStream_t s = (hipStream_t)stream;
  if (a->n_split == 0 || a->vdimp > 128 || a->dimp > 128 || !mix_fast(a->H, a->G, a->dim, a->vdim, a->f32)) return p3v_attn_mix_any(a, s);
  if (a->n_split > 1 && (!a->ws || a->n_split > MIX_MAX_ROW_SPLIT)) return P3V_ERR_ARG;
  AttnMixP p = attn_mix_params(a);
  // (the position may be a device value: the splits then cover the capacity)
  p.tiles_per_split = p3v_cdiv(p3v_cdiv(a->d_past ? a->Tp : a->past + a->L, 32), a->n_split);
  if (p.n_split > 1 && p.L == 1) return P3V_ERR_ARG;                     // (k_attn_mix_combine's splits are 16-key tiles)
  const int per = p.H / p.G;                                             // query heads of a key / value head
  if (p.H <= 8) return prefill_dc<1, true>(p, s);
  if (p.H <= 16) return per % 2 ? prefill_dc<2, false>(p, s) : prefill_dc<2, true>(p, s);
  return per % 4 ? prefill_dc<4, false>(p, s) : prefill_dc<4, true>(p, s);
}

template <int GW, int DC, int NP>
static int launch_decode(const QkvHeadsP& hp, const AttnMixP& p, hipStream_t s) {
  const bool vec = p.dim % 8 == 0 && p.vdim % 8 == 0 && hp.ld % 8 == 0 && (!hp.v_first || hp.ld_first % 8 == 0) && p.H * p.dim <= 4096 &&
                   (((uintptr_t)hp.qkv | (uintptr_t)hp.q_norm | (uintptr_t)hp.k_norm | (uintptr_t)hp.v_first) & 15) == 0;
  const dim3 grid(p.n_split, p.B);
  const size_t lds = (size_t)p.H * p.dimp * 2;
  if (vec) hipLaunchKernelGGL((k_attn_mix_decode<GW, DC, NP, true>), grid, dim3(512), lds, s, hp, p);
  else hipLaunchKernelGGL((k_attn_mix_decode<GW, DC, NP, false>), grid, dim3(512), lds, s, hp, p);
  P3V_CHECK_LAUNCH();
  return mix_combine(p, s);
}
template <int GW, int DC>
static int decode_np(const QkvHeadsP& hp, const AttnMixP& p, hipStream_t s) {
  const int np = p3v_cdiv(p.H * p.vdim, 512);
  return np <= 2 ? launch_decode<GW, DC, 2>(hp, p, s) : np <= 4 ? launch_decode<GW, DC, 4>(hp, p, s)
       : np <= 6 ? launch_decode<GW, DC, 6>(hp, p, s) : launch_decode<GW, DC, 8>(hp, p, s);
}
template <int DC>
static int decode_gw(const QkvHeadsP& hp, const AttnMixP& p, hipStream_t s) {
  return p.G <= 8 ? decode_np<1, DC>(hp, p, s) : p.G <= 16 ? decode_np<2, DC>(hp, p, s) : decode_np<4, DC>(hp, p, s);
}

extern "C" int p3v_attn_mix_decode(const p3v_mix_args_t* a, void* stream) {
  const int rc = p3v_mix_check(a);
  if (rc != P3V_OK) return rc;
  if (!a->qkv || !a->q_norm || !a->k_norm || !a->talk || !a->sink || !a->gate || !a->out || a->n_split < 0) return P3V_ERR_ARG;
  if (a->L != 1 || a->n_split == 0 || !mix_fast(a->H, a->G, a->dim, a->vdim, a->f32) || a->H / a->G > 16 || a->dimp > 128)
    return P3V_ERR_UNSUPPORTED;
  if (!a->ws || a->n_split > MIX_MAX_SPLIT) return P3V_ERR_ARG;
  AttnMixP p = attn_mix_params(a);
  p.tiles_per_split = p3v_cdiv(a->Tp / 16, a->n_split);
  const QkvHeadsP hp = {a->qkv, a->q_norm, a->k_norm, a->v_first, nullptr, a->k, a->v, a->d_past, a->eps, a->vmix,
                        a->B, a->L, a->H, a->G, a->dim, a->vdim, a->dimp, a->vdimp, a->ld, a->ld_first, a->past, a->Tp};
  hipStream_t s = (hipStream_t)stream;
  switch (a->dimp / 32) {
    case 1: return decode_gw<1>(hp, p, s);
    case 2: return decode_gw<2>(hp, p, s);
    case 3: return decode_gw<3>(hp, p, s);
    default: return decode_gw<4>(hp, p, s);
  }
}
