// Several residual streams (hyper-connections): the row kernel at every sublayer boundary.
//   x_t <- sum_s mix[s][t] x_s + out[t] y        (all t from the old streams; f32)
//   u    = sum_s in[s] x_s,   xn = u / sqrt(mean(u^2) + eps) * norm_w
// One pass over the streams per boundary: the update by the sublayer that has just run and the input of the next one
// are the same launch.  The first boundary of a pass fills the streams from the embedding (+ position vector), the
// last one (store == 0) only makes the normed sum.
#include "tmx_kernels.h"

namespace tmx {

__device__ __forceinline__ float4 act4(const uint16_t* p) {
  const uint2 v = *reinterpret_cast<const uint2*>(p);
  return make_float4(bf_lo(v.x), bf_hi(v.x), bf_lo(v.y), bf_hi(v.y));
}
__device__ __forceinline__ float4 act4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ void put_act4(uint16_t* p, float4 v) {
  *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf2(v.x, v.y), pack_bf2(v.z, v.w));
}
__device__ __forceinline__ void put_act4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
__device__ __forceinline__ void fma4(float4& d, float c, const float4& x) {
  d.x = fmaf(c, x.x, d.x); d.y = fmaf(c, x.y, d.y); d.z = fmaf(c, x.z, d.z); d.w = fmaf(c, x.w, d.w);
}

// One workgroup per row; a thread owns 4 consecutive columns at a time, u waits in LDS for the root mean square.
template <int S, typename T, int NTH>
__global__ __launch_bounds__(NTH) void stream_rows_kernel(StreamArgs a) {
  extern __shared__ __align__(16) float u_s[];  // [Dp]
  __shared__ float smem[NTH / 64];
  const int m = blockIdx.x;
  float* xs = a.xs + (size_t)m * S * a.Dp;
  const T* y = a.y ? reinterpret_cast<const T*>(a.y) + (size_t)m * a.Dp : nullptr;
  const bool upd = y || a.y_part;
  const uint16_t *er = nullptr, *pr = nullptr;
  if (a.embed) {
    const int tpp = a.tpp > 0 ? a.tpp : 1;
    const int seq = m / tpp, col = min(*a.step + m % tpp, a.buf_len - 1);
    const int tok = min(max(a.token_buffer[(size_t)seq * a.buf_len + col], 0), a.vocab - 1);
    er = a.embed + (size_t)tok * a.Dp;
    if (a.pos_embed) {
      const int pos = min(max(a.positions[(size_t)seq * a.buf_len + col], 0), a.max_positions - 1);
      pr = a.pos_embed + (size_t)pos * a.Dp;
    }
  }
  float ci[S], co[S], cm[S][S];
#pragma unroll
  for (int s = 0; s < S; ++s) {
    ci[s] = a.in[s];
    co[s] = upd ? a.out[s] : 0.f;
#pragma unroll
    for (int t = 0; t < S; ++t) cm[s][t] = upd ? a.mix[s * S + t] : 0.f;
  }
  float ss = 0.f;
#pragma unroll 2
  for (int c = threadIdx.x * 4; c < a.Dp; c += NTH * 4) {
    float4 x[S];
    if (er) {
      float4 e = act4(er + c);
      if (pr) {
        const float4 p = act4(pr + c);
        e.x += p.x; e.y += p.y; e.z += p.z; e.w += p.w;
      }
#pragma unroll
      for (int s = 0; s < S; ++s) x[s] = e;
    } else {
#pragma unroll
      for (int s = 0; s < S; ++s) x[s] = *reinterpret_cast<const float4*>(xs + (size_t)s * a.Dp + c);
    }
    if (upd) {
      float4 yv;
      if (a.y_part) {  // planes in ascending order, all requested before the first add
        float4 pl[4];
#pragma unroll
        for (int i = 0; i < 4; ++i)
          pl[i] = *reinterpret_cast<const float4*>(a.y_part + ((size_t)min(i, a.nsplit - 1) * gridDim.x + m) * a.Dp + c);
        yv = pl[0];
#pragma unroll
        for (int i = 1; i < 4; ++i)
          if (i < a.nsplit) { yv.x += pl[i].x; yv.y += pl[i].y; yv.z += pl[i].z; yv.w += pl[i].w; }
      } else {
        yv = act4(y + c);
      }
      float4 old[S];
#pragma unroll
      for (int s = 0; s < S; ++s) old[s] = x[s];
#pragma unroll
      for (int t = 0; t < S; ++t) {
        x[t] = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int s = 0; s < S; ++s) fma4(x[t], cm[s][t], old[s]);
        fma4(x[t], co[t], yv);
      }
    }
    float4 u = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int s = 0; s < S; ++s) {
      fma4(u, ci[s], x[s]);
      if (a.store && (er || upd)) *reinterpret_cast<float4*>(xs + (size_t)s * a.Dp + c) = x[s];
    }
    *reinterpret_cast<float4*>(u_s + c) = u;
    ss += u.x * u.x + u.y * u.y + u.z * u.z + u.w * u.w;
  }
  ss = block_sum<NTH / 64>(ss, smem);
  const float inv = 1.f / sqrtf(ss / (float)a.D + a.eps);
  T* xn = reinterpret_cast<T*>(a.xn);
  for (int c = threadIdx.x * 4; c < a.Dp; c += NTH * 4) {
    const float4 u = *reinterpret_cast<const float4*>(u_s + c), w = *reinterpret_cast<const float4*>(a.norm_w + c);
    put_act4(xn + (a.xn_tiled ? act_tile_off(m, c, a.Dp) : (size_t)m * a.Dp + c), make_float4(u.x * inv * w.x, u.y * inv * w.y, u.z * inv * w.z, u.w * inv * w.w));
  }
}

template <int S, typename T>
static void launch_streams(hipStream_t st, const StreamArgs& a, int M) {
  const size_t lds = (size_t)a.Dp * 4;
  if (a.Dp >= 2048) hipLaunchKernelGGL((stream_rows_kernel<S, T, 512>), dim3(M), dim3(512), lds, st, a);
  else hipLaunchKernelGGL((stream_rows_kernel<S, T, 256>), dim3(M), dim3(256), lds, st, a);
}

int stream_rows(hipStream_t st, int act, const StreamArgs& a, int M) {
  if (M <= 0 || a.Dp <= 0 || a.Dp % 64 || a.D > a.Dp || a.D <= 0 || a.Dp > 14336) return TMX_ERR_SHAPE;
  if (act != TMX_ACT_BF16 && act != TMX_ACT_F32) return TMX_ERR_ARG;
  if (a.y_part && (a.nsplit < 1 || a.nsplit > 4)) return TMX_ERR_ARG;
#define TMX_STREAMS(n)                                           \
  case n:                                                        \
    if (act == TMX_ACT_BF16) launch_streams<n, uint16_t>(st, a, M); \
    else launch_streams<n, float>(st, a, M);                     \
    break;
  switch (a.S) {
    TMX_STREAMS(1) TMX_STREAMS(2) TMX_STREAMS(3) TMX_STREAMS(4)
    TMX_STREAMS(5) TMX_STREAMS(6) TMX_STREAMS(7) TMX_STREAMS(8)
    default: return TMX_ERR_SHAPE;
  }
#undef TMX_STREAMS
  return check_launch();
}

}  // namespace tmx

using namespace tmx;

extern "C" int tmx_stream_rows(void* stream, int act, float* streams, const void* y, const float* mix,
                               const float* out, const float* in, const float* norm_w, void* xn, int M, int S, int D,
                               int Dp, float eps, int store) {
  if (!streams || !in || !norm_w || !xn || (y && (!mix || !out))) return TMX_ERR_ARG;
  StreamArgs a = {};
  a.xs = streams; a.y = y; a.mix = mix; a.out = out; a.in = in; a.norm_w = norm_w; a.xn = xn;
  a.S = S; a.D = D; a.Dp = Dp; a.eps = eps; a.store = store;
  return stream_rows((hipStream_t)stream, act, a, M);
}
