// Row part of latent attention in front of the walk: rotation of the queries, norm + rotation of the new cache row.
// A launch of its own (latent.hip), or extra workgroups of the launch that moves the queries into the latent space
// (dense.hip): the two write different columns of the query tensor.
#pragma once
#include "tmx_kernels.h"

namespace tmx {

__device__ __forceinline__ float act_get(const uint16_t* p) { return bf2f(*p); }
__device__ __forceinline__ float act_get(const float* p) { return *p; }
__device__ __forceinline__ void act_set(uint16_t* p, float v) { *p = f2bf(v); }
__device__ __forceinline__ void act_set(float* p, float v) { *p = v; }

// One workgroup of NTH threads per row m of the fused projection; smem: NTH / 64 floats.
template <typename T, int NTH>
__device__ __forceinline__ void latent_rows_block(const LatentRowsArgs& a, int m, float* smem) {
  constexpr int VP = TMX_MAX_LATENT_RANK / NTH;  // latent values per thread
  const int tid = threadIdx.x;
  const int tpp = a.tpp > 0 ? a.tpp : 1;
  const int seq = m / tpp, slot = min(*a.step + m % tpp, min(a.buf_len, a.C) - 1);
  const int pos = min(max(a.positions[(size_t)seq * a.buf_len + slot], 0), a.max_positions - 1);
  const int half = a.rot >> 1, ld = a.rank_p + a.rot_p;
  const float2* tab = reinterpret_cast<const float2*>(a.table) + (size_t)pos * half;
  const T* z = reinterpret_cast<const T*>(a.z) + (size_t)m * a.ldz;
  T* q = reinterpret_cast<T*>(a.q) + (size_t)m * a.H * ld + a.rank_p;
  float v[VP] = {};
  if (a.off_kv >= 0) {
#pragma unroll
    for (int i = 0; i < VP; ++i)
      if (tid + NTH * i < a.rank) v[i] = act_get(z + a.off_kv + tid + NTH * i);
  }
  // rotated query part of every head; columns from the real width on are zero
  for (int e = tid; e < a.H * half; e += NTH) {
    const int hd = e / half, i = e - hd * half;
    const float u = act_get(z + a.off_qr + hd * a.rot + i), w = act_get(z + a.off_qr + hd * a.rot + half + i);
    const float2 cs = tab[i];
    act_set(q + (size_t)hd * ld + i, u * cs.x - w * cs.y);
    act_set(q + (size_t)hd * ld + half + i, w * cs.x + u * cs.y);
  }
  const int pad = a.rot_p - a.rot;
  for (int e = tid; e < a.H * pad; e += NTH) act_set(q + (size_t)(e / pad) * ld + a.rot + e % pad, 0.f);
  if (a.off_kv < 0) return;
  T* row = reinterpret_cast<T*>(a.cache) + ((size_t)seq * a.C + slot) * ld;
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < VP; ++i) ss += v[i] * v[i];
  ss = block_sum<NTH / 64>(ss, smem);
  const float inv = 1.f / sqrtf(ss / (float)a.rank + a.eps);
#pragma unroll
  for (int i = 0; i < VP; ++i) {
    const int c = tid + NTH * i;
    if (c < a.rank_p) act_set(row + c, c < a.rank ? v[i] * inv * a.norm_w[c] : 0.f);
  }
  if (tid < a.rot_p) {
    float o = 0.f;
    if (tid < a.rot) {
      const T* kr = z + a.off_kv + a.rank;
      const int i = tid < half ? tid : tid - half;
      const float u = act_get(kr + i), w = act_get(kr + half + i);
      const float2 cs = tab[i];
      o = tid < half ? u * cs.x - w * cs.y : w * cs.x + u * cs.y;
    }
    act_set(row + a.rank_p + tid, o);
  }
}

}  // namespace tmx
