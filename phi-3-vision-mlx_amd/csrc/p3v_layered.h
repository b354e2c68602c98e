// Shared by the kernels of the layered text decoders (p3v_layered.hip, p3v_attn_mix.hip, the fused prologue of p3v_gemv.hip).
#pragma once
#include "p3v_common.h"

// ---- activations: bf16 or fp32 in memory, fp32 in registers
__device__ __forceinline__ float load_act(const bf16_t* p) { return bf16_to_f32(*p); }
__device__ __forceinline__ float load_act(const float* p) { return *p; }
__device__ __forceinline__ void store_act(bf16_t* p, float v) { *p = f32_to_bf16(v); }
__device__ __forceinline__ void store_act(float* p, float v) { *p = v; }
template <typename T> __device__ __forceinline__ float round_act(float v);
template <> __device__ __forceinline__ float round_act<bf16_t>(float v) { return bf16_round(v); }
template <> __device__ __forceinline__ float round_act<float>(float v) { return v; }
// V consecutive activations; V = 8 needs 16-byte aligned addresses
template <int V> __device__ __forceinline__ void load_acts(const bf16_t* p, float* v) {
  if constexpr (V == 8) {
    const u32x4_t w = *(const u32x4_t*)p;
#pragma unroll
    for (int j = 0; j < 4; ++j) v[2 * j] = bf16lo(w[j]), v[2 * j + 1] = bf16hi(w[j]);
  } else {
    v[0] = load_act(p);
  }
}
template <int V> __device__ __forceinline__ void load_acts(const float* p, float* v) {
  if constexpr (V == 8) {
    const float4 a = *(const float4*)p, b = *(const float4*)(p + 4);
    v[0] = a.x, v[1] = a.y, v[2] = a.z, v[3] = a.w, v[4] = b.x, v[5] = b.y, v[6] = b.z, v[7] = b.w;
  } else {
    v[0] = *p;
  }
}
template <int V> __device__ __forceinline__ void store_acts(bf16_t* p, const float* v) {
  if constexpr (V == 8) {
    u32x4_t w;
#pragma unroll
    for (int j = 0; j < 4; ++j) w[j] = pack_bf16x2(v[2 * j], v[2 * j + 1]);
    *(u32x4_t*)p = w;
  } else {
    store_act(p, v[0]);
  }
}
template <int V> __device__ __forceinline__ void store_acts(float* p, const float* v) {
  if constexpr (V == 8) {
    *(float4*)p = make_float4(v[0], v[1], v[2], v[3]);
    *(float4*)(p + 4) = make_float4(v[4], v[5], v[6], v[7]);
  } else {
    *p = v[0];
  }
}

// four consecutive ones, 8-byte (bf16) or 16-byte (fp32) aligned
__device__ __forceinline__ void load4(const bf16_t* p, float (&v)[4]) {
  const u32x2_t w = *(const u32x2_t*)p;
  v[0] = bf16lo(w[0]), v[1] = bf16hi(w[0]), v[2] = bf16lo(w[1]), v[3] = bf16hi(w[1]);
}
__device__ __forceinline__ void load4(const float* p, float (&v)[4]) {
  const float4 w = *(const float4*)p;
  v[0] = w.x, v[1] = w.y, v[2] = w.z, v[3] = w.w;
}
__device__ __forceinline__ void store4(bf16_t* p, const float (&v)[4]) { *(u32x2_t*)p = (u32x2_t){pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3])}; }
__device__ __forceinline__ void store4(float* p, const float (&v)[4]) { *(float4*)p = make_float4(v[0], v[1], v[2], v[3]); }

// ---- kernel parameters
struct DytP {
  const float* x; const bf16_t* w; const bf16_t* b; const bf16_t* mu; float* hist; const int32_t* pad_len; const int32_t* d_past;
  float alpha; int past, R, B, L, H;
};
static inline DytP dyt_params(const p3v_dyt_args_t* a) {
  return {a->x, a->w, a->b, a->mu, a->hist, a->pad_len, a->d_past, a->alpha, a->past, a->hist_rows, a->B, a->L, a->H};
}
struct QkvHeadsP {
  const void* qkv; const bf16_t* q_norm; const bf16_t* k_norm; const void* v_first; void* q; void* k; void* v; const int32_t* d_past;
  float eps, vmix; int B, L, H, G, dim, vdim, dimp, vdimp, ld, ld_first, past, Tp;
};
struct AttnMixP {
  const void* q; const void* k; const void* v; const bf16_t* talk; const bf16_t* sink; const void* gate; void* out; float* ws;
  const int32_t* pad_len; const int32_t* d_past;
  float scale; int B, L, H, G, dim, vdim, dimp, vdimp, ld, past, Tp, n_split, tiles_per_split;
};
static inline AttnMixP attn_mix_params(const p3v_mix_args_t* a) {
  return {a->q, a->k, a->v, a->talk, a->sink, a->gate, a->out, a->ws, a->pad_len, a->d_past, a->scale,
          a->B, a->L, a->H, a->G, a->dim, a->vdim, a->dimp, a->vdimp, a->ld, a->past, a->Tp, a->n_split, 0};
}

int p3v_dyt_check(const p3v_dyt_args_t* a);
int p3v_mix_check(const p3v_mix_args_t* a);
int p3v_attn_mix_any(const p3v_mix_args_t* a, hipStream_t s);
