// Latent attention: shared by p3v_latent.hip (append, attention in the latent space) and p3v_latent_prompt.hip (over expanded keys).
#pragma once
#include "p3v_layered.h"

#define LAT_NEG (-1e30f)             // "no key yet": finite, so that differences of two of them stay 0
#define LAT_LOG2E 1.4426950408889634f

struct LatP {
  void* y; const bf16_t* c_norm; const bf16_t* uk; const bf16_t* ukt; const bf16_t* uv; const bf16_t* sink;
  const float* cos_t; const float* sin_t; void* c; void* q; const void* kx; const void* vx; void* out; float* ws;
  const int32_t* pad_len; const int32_t* d_past;
  float eps, scale;
  int B, L, H, dim, rot, vdim, rank, rankp, rotp, dimp, ld, past, Tp, tab_n, n_keys, n_split, tiles_per_split;
};
static inline LatP lat_params(const p3v_latent_args_t* a) {
  return {a->y, a->c_norm, a->uk, a->ukt, a->uv, a->sink, a->cos_t, a->sin_t, a->c, a->q, a->kx, a->vx, a->out, a->ws, a->pad_len, a->d_past,
          a->eps, a->scale, a->B, a->L, a->H, a->dim, a->rot, a->vdim, a->rank, a->rankp, a->rotp, a->dimp, a->ld, a->past, a->Tp, a->tab_n,
          a->n_keys, a->n_split, 0};
}
// first columns of a packed row
__host__ __device__ __forceinline__ int lat_dkv_col(const LatP& p) { return p.H * (p.dim + p.rot); }
__host__ __device__ __forceinline__ int lat_gate_col(const LatP& p) { return lat_dkv_col(p) + p.rank + p.rot; }

__device__ __forceinline__ float lat_gate(float z) { return 1.f / (1.f + expf(-z)); }
// workgroup barrier for LDS data only: global loads stay in flight across it
__device__ __forceinline__ void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}

int p3v_latent_check(const p3v_latent_args_t* a);
bool p3v_latent_prompt_fits(int dim, int rot, int vdim);
