// Latent attention of a prompt, over keys and values expanded once per call (kx [B, n_keys, H dim] = latents x uk, vx [B, H vdim, n_keys] =
// uv x latents: two plain matrix products); the rotated key part comes from the cache.
//
// A workgroup: one head, 128 queries, 32 per wave, tiles of 64 keys in LDS (requested a tile ahead into registers).  Scores are computed
// transposed, keys x queries, on 32 x 32 x 16 MFMAs: a lane then holds 16 keys of ONE query, the softmax is lane-local but for one exchange
// between the two halves of the wave, and the probabilities are the second product's operand as they lie -- of the 16 keys of a step a
// half holds {0..3, 8..11} + 4 half, and the value fragments are read in that order.
#include "p3v_latent.h"

template <int KC, int VT> struct PromptCfg {                              // KC: 16-dimension chunks of a key, VT: 32-dimension tiles of a value
  static constexpr int KS = KC * 16 + 8, VS = 72, K = 64 * KS * 2, V = VT * 32 * VS * 2, LDS = K + V;
  static constexpr int NK = KC / 2, NV = VT;                              // 16-byte pieces per thread of a tile
};

template <int KC, int VT>
__global__ void __launch_bounds__(256, KC * 4 + VT * 16 <= 112 && (KC <= 12 || VT <= 2) ? 2 : 1) k_latent_prompt(LatP p) {
  typedef PromptCfg<KC, VT> C;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  bf16_t *Ks = (bf16_t*)smem, *Vs = (bf16_t*)(smem + C::K);
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lc = lane & 31, lg = lane >> 5;
  const int h = blockIdx.x, q0 = ((int)gridDim.y - 1 - (int)blockIdx.y) * 128, b = blockIdx.z;             // longest rows first
  const int past = p.d_past ? *p.d_past : p.past, first = p.pad_len ? p.pad_len[b] : 0;
  const int DC = (p.dim + 15) / 16, W = p.dim + p.rot, QW = p.rankp + p.rotp;
  const int wq0 = q0 + wave * 32, wlast = past + min(wq0 + 31, p.L - 1), last = past + min(q0 + 127, p.L - 1);
  const int t0 = first >> 6, t1 = (last >> 6) + 1;
  const float sc = fabsf(p.scale) * LAT_LOG2E;                            // (a negative scale's sign goes into the queries: the row maxima then scale)
  const uint32_t flip = p.scale < 0.f ? 0x80008000u : 0u;

  // queries (B operand: column = query, 8 consecutive dimensions)
  bf16x8_t qf[KC];
  {
    const bf16_t* q = (const bf16_t*)p.y + ((size_t)b * p.L + min(wq0 + lc, p.L - 1)) * p.ld + h * W;
#pragma unroll
    for (int c = 0; c < KC; ++c) {
      const bool nope = c < DC;
      const int d = (nope ? c : c - DC) * 16 + lg * 8;
      u32x4_t v = {0u, 0u, 0u, 0u};
      if (d < (nope ? p.dim : p.rot)) v = *(const u32x4_t*)(q + (nope ? d : p.dim + d));
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] ^= flip;
      qf[c] = __builtin_bit_cast(bf16x8_t, v);
    }
  }
  // this thread's pieces of a tile: keys row by row, values dimension by dimension; pieces of no dimension are zero
  const bf16_t* ksrc[C::NK];
  uint32_t kstep[C::NK];
  const bf16_t* vsrc[C::NV];
#pragma unroll
  for (int i = 0; i < C::NK; ++i) {
    const int e = tid + 256 * i, key = e / (2 * KC), part = e - key * (2 * KC);
    const bool nope = part < 2 * DC;
    const int d = (nope ? part : part - 2 * DC) * 8;
    ksrc[i] = nullptr, kstep[i] = 0;
    if (nope && d < p.dim) ksrc[i] = (const bf16_t*)p.kx + ((size_t)b * p.n_keys + key) * p.H * p.dim + h * p.dim + d, kstep[i] = 64 * p.H * p.dim;
    if (!nope && d < p.rot) ksrc[i] = (const bf16_t*)p.c + ((size_t)b * p.Tp + key) * QW + p.rankp + d, kstep[i] = 64 * QW;
  }
#pragma unroll
  for (int i = 0; i < C::NV; ++i) {
    const int e = tid + 256 * i, v = e >> 3;
    vsrc[i] = v < p.vdim ? (const bf16_t*)p.vx + (((size_t)b * p.H + h) * p.vdim + v) * p.n_keys + (e & 7) * 8 : nullptr;
  }
  u32x4_t kr[C::NK], vr[C::NV];
  constexpr u32x4_t zero4 = {0u, 0u, 0u, 0u};
  auto load = [&](int t) {
#pragma unroll
    for (int i = 0; i < C::NK; ++i) kr[i] = ksrc[i] ? *(const u32x4_t*)(ksrc[i] + (size_t)t * kstep[i]) : zero4;
#pragma unroll
    for (int i = 0; i < C::NV; ++i) vr[i] = vsrc[i] ? *(const u32x4_t*)(vsrc[i] + (size_t)t * 64) : zero4;
  };

  f32x16_t o[VT];
#pragma unroll
  for (int v = 0; v < VT; ++v)
#pragma unroll
    for (int i = 0; i < 16; ++i) o[v][i] = 0.f;
  float m_run = LAT_NEG, l_run = 0.f;                                     // of query lc; the sum over this half's keys
  if (t0 < t1) load(t0);
  for (int t = t0; t < t1; ++t) {
    lds_barrier();                                                        // (everybody is done with the tile before)
#pragma unroll
    for (int i = 0; i < C::NK; ++i) { const int e = tid + 256 * i, key = e / (2 * KC); *(u32x4_t*)(Ks + key * C::KS + (e - key * (2 * KC)) * 8) = kr[i]; }
#pragma unroll
    for (int i = 0; i < C::NV; ++i) { const int e = tid + 256 * i; *(u32x4_t*)(Vs + (e >> 3) * C::VS + (e & 7) * 8) = vr[i]; }
    if (t + 1 < t1) load(t + 1);
    lds_barrier();
    if (t * 64 > wlast) continue;                                         // (no query of this wave sees the tile)
    f32x16_t s[2];
#pragma unroll
    for (int k = 0; k < 2; ++k) {
#pragma unroll
      for (int i = 0; i < 16; ++i) s[k][i] = 0.f;
#pragma unroll
      for (int c = 0; c < KC; ++c)
        s[k] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*(const bf16x8_t*)(Ks + (k * 32 + lc) * C::KS + c * 16 + lg * 8), qf[c], s[k], 0, 0, 0);
    }
    if (t * 64 + 63 > past + wq0 || t * 64 < first) {
      const int qpos = past + wq0 + lc;
#pragma unroll
      for (int k = 0; k < 2; ++k)
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          const int key = t * 64 + k * 32 + 8 * (i >> 2) + 4 * lg + (i & 3);
          s[k][i] = key <= qpos && key >= first ? s[k][i] : -INFINITY;
        }
    }
    float mx = fmaxf(s[0][0], s[1][0]);
#pragma unroll
    for (int i = 1; i < 16; ++i) mx = fmaxf(mx, fmaxf(s[0][i], s[1][i]));
    float xa, xb;
    rows_swap32(mx, xa, xb);
    const float mn = fmaxf(m_run, fmaxf(xa, xb) * sc);
    if (__builtin_amdgcn_ballot_w64(mn != m_run)) {                       // (a maximum moved; rare behind a sequence's first tiles)
      const float al = __builtin_amdgcn_exp2f(m_run - mn);
      l_run *= al;
#pragma unroll
      for (int v = 0; v < VT; ++v) o[v] *= al;
      m_run = mn;
    }
    bf16x8_t pf[2][2];
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      float ls = 0.f;
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        s[k][i] = __builtin_amdgcn_exp2f(fmaf(s[k][i], sc, -m_run));
        ls += s[k][i];
      }
      l_run += ls;
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        u32x4_t w;
#pragma unroll
        for (int j = 0; j < 4; ++j) w[j] = pack_bf16x2(s[k][8 * u + 2 * j], s[k][8 * u + 2 * j + 1]);
        pf[k][u] = __builtin_bit_cast(bf16x8_t, w);
      }
    }
#pragma unroll
    for (int k = 0; k < 2; ++k)
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        const bf16_t* vp = Vs + lc * C::VS + k * 32 + u * 16 + lg * 4;
#pragma unroll
        for (int v = 0; v < VT; ++v) {
          const u32x2_t a = *(const u32x2_t*)(vp + v * 32 * C::VS), c = *(const u32x2_t*)(vp + v * 32 * C::VS + 8);
          const u32x4_t w = {a[0], a[1], c[0], c[1]};
          o[v] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, w), pf[k][u], o[v], 0, 0, 0);
        }
      }
  }
  float la, lb;
  rows_swap32(l_run, la, lb);
  const int l = wq0 + lc;
  if (l >= p.L) return;
  const float sk = bf16_to_f32(p.sink[h]) * LAT_LOG2E, mm = fmaxf(m_run, sk), e = __builtin_amdgcn_exp2f(m_run - mm);
  const float f = e / ((la + lb) * e + __builtin_amdgcn_exp2f(sk - mm));
  const size_t row = (size_t)b * p.L + l;
  const bf16_t* gate = (const bf16_t*)p.y + row * p.ld + lat_gate_col(p) + h * p.vdim;
  bf16_t* out = (bf16_t*)p.out + row * p.H * p.vdim + (size_t)h * p.vdim;
#pragma unroll
  for (int v = 0; v < VT; ++v)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int c = v * 32 + 8 * i + 4 * lg;
      if (c < p.vdim) {
        const u32x2_t z = *(const u32x2_t*)(gate + c);
        float g[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) g[r] = o[v][4 * i + r] * f * p3v_sigmoid(r & 1 ? bf16hi(z[r >> 1]) : bf16lo(z[r >> 1]));
        *(u32x2_t*)(out + c) = (u32x2_t){pack_bf16x2(g[0], g[1]), pack_bf16x2(g[2], g[3])};
      }
    }
}

template <int KC, int VT> static int launch_prompt(const LatP& p, hipStream_t s) {
  constexpr int lds = PromptCfg<KC, VT>::LDS;
  static bool set = false;
  if (!set) {
    if (hipFuncSetAttribute((const void*)k_latent_prompt<KC, VT>, hipFuncAttributeMaxDynamicSharedMemorySize, lds) != hipSuccess) return P3V_ERR_HIP;
    set = true;
  }
  // heads innermost: with a multiple of 8 of them a head's workgroups stay on one XCD, whose L2 holds its keys
  hipLaunchKernelGGL((k_latent_prompt<KC, VT>), dim3(p.H, p3v_cdiv(p.L, 128), p.B), dim3(256), lds, s, p);
  P3V_CHECK_LAUNCH();
  return P3V_OK;
}
template <int KC> static int prompt_vt(const LatP& p, hipStream_t s) {
  const int vt = p3v_cdiv(p.vdim, 32);
  return vt <= 2 ? launch_prompt<KC, 2>(p, s) : vt <= 3 ? launch_prompt<KC, 3>(p, s) : vt <= 4 ? launch_prompt<KC, 4>(p, s) : launch_prompt<KC, 8>(p, s);
}
static int prompt_kc(int dim, int rot) { return p3v_cdiv(dim, 16) + p3v_cdiv(rot, 16); }
bool p3v_latent_prompt_fits(int dim, int rot, int vdim) { return dim % 8 == 0 && rot % 8 == 0 && vdim % 8 == 0 && prompt_kc(dim, rot) <= 16 && vdim <= 256; }

extern "C" int p3v_latent_prompt(const p3v_latent_args_t* a, void* stream) {
  const int rc = p3v_latent_check(a);
  if (rc != P3V_OK) return rc;
  if (!a->kx || !a->vx || !a->out || a->n_keys % 64 || a->n_keys > a->Tp || (!a->d_past && a->past + a->L > a->n_keys)) return P3V_ERR_ARG;
  if (a->f32 || !p3v_latent_prompt_fits(a->dim, a->rot, a->vdim) || a->rank % 8 || a->ld % 8 || a->B > 65535) return P3V_ERR_UNSUPPORTED;
  if (((uintptr_t)a->y | (uintptr_t)a->kx | (uintptr_t)a->vx | (uintptr_t)a->c | (uintptr_t)a->out) & 15) return P3V_ERR_ARG;
  const LatP p = lat_params(a);
  hipStream_t s = (hipStream_t)stream;
  const int kc = prompt_kc(a->dim, a->rot);
  return kc <= 4 ? prompt_vt<4>(p, s) : kc <= 6 ? prompt_vt<6>(p, s) : kc <= 8 ? prompt_vt<8>(p, s) : kc <= 12 ? prompt_vt<12>(p, s) : prompt_vt<16>(p, s);
}
