// Row kernels at the sublayer boundaries of dense models.  Several residual streams (hyper-connections):
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
      e.x *= a.embed_scale; e.y *= a.embed_scale; e.z *= a.embed_scale; e.w *= a.embed_scale;
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

// ---------------------------------------------------------------------------
// One residual stream, the norm behind the sublayer and / or in front of the next one (tmx_residual_rows).  A thread keeps
// its NC groups of 4 columns in registers; the two root mean squares are the only exchange.
template <typename T, int NTH, int NC>
__global__ __launch_bounds__(NTH) void residual_rows_kernel(ResidualArgs a) {
  __shared__ float smem[2][NTH / 64];
  const int m = blockIdx.x;
  float* xr = a.x + (size_t)m * a.Dp;
  const bool upd = a.y || a.y_part;
  const uint16_t* er = nullptr;
  if (a.embed) {
    const int tpp = a.tpp > 0 ? a.tpp : 1;
    const int col = min(*a.step + m % tpp, a.buf_len - 1);
    const int tok = min(max(a.token_buffer[(size_t)(m / tpp) * a.buf_len + col], 0), a.vocab - 1);
    er = a.embed + (size_t)tok * a.Dp;
  }
  float4 x[NC], y[NC];
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = ((int)threadIdx.x + i * NTH) * 4;
    x[i] = y[i] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (c >= a.Dp) continue;
    if (er) {
      const float4 e = act4(er + c);
      x[i] = make_float4(e.x * a.embed_scale, e.y * a.embed_scale, e.z * a.embed_scale, e.w * a.embed_scale);
    } else {
      x[i] = *reinterpret_cast<const float4*>(xr + c);
    }
    if (a.y_part) {  // planes in ascending order, all requested before the first add
      float4 pl[4];
#pragma unroll
      for (int k = 0; k < 4; ++k)
        pl[k] = *reinterpret_cast<const float4*>(a.y_part + ((size_t)min(k, a.nsplit - 1) * gridDim.x + m) * a.Dp + c);
      y[i] = pl[0];
#pragma unroll
      for (int k = 1; k < 4; ++k)
        if (k < a.nsplit) { y[i].x += pl[k].x; y[i].y += pl[k].y; y[i].z += pl[k].z; y[i].w += pl[k].w; }
    } else if (a.y) {
      y[i] = act4(reinterpret_cast<const T*>(a.y) + (size_t)m * a.Dp + c);
    }
  }
  auto inverse_rms = [&](const float4* v, float* area) __attribute__((always_inline)) {
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NC; ++i) ss += v[i].x * v[i].x + v[i].y * v[i].y + v[i].z * v[i].z + v[i].w * v[i].w;
    return 1.f / sqrtf(block_sum<NTH / 64>(ss, area) / (float)a.D + a.eps);
  };
  const bool post = upd && a.post_w;
  const float py = post ? inverse_rms(y, smem[0]) : 1.f;
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = ((int)threadIdx.x + i * NTH) * 4;
    if (c >= a.Dp) continue;
    if (upd) {
      const float4 w = post ? *reinterpret_cast<const float4*>(a.post_w + c) : make_float4(1.f, 1.f, 1.f, 1.f);
      x[i].x += y[i].x * py * w.x; x[i].y += y[i].y * py * w.y;
      x[i].z += y[i].z * py * w.z; x[i].w += y[i].w * py * w.w;
    }
    if (a.store && (er || upd)) *reinterpret_cast<float4*>(xr + c) = x[i];
  }
  const float nx = a.norm_w ? inverse_rms(x, smem[1]) : 1.f;
  T* xn = reinterpret_cast<T*>(a.xn);
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = ((int)threadIdx.x + i * NTH) * 4;
    if (c >= a.Dp) continue;
    float4 v = x[i];
    if (a.norm_w) {
      const float4 w = *reinterpret_cast<const float4*>(a.norm_w + c);
      v = make_float4(v.x * nx * w.x, v.y * nx * w.y, v.z * nx * w.z, v.w * nx * w.w);
    }
    put_act4(xn + (a.xn_tiled ? act_tile_off(m, c, a.Dp) : (size_t)m * a.Dp + c), v);
  }
}

template <typename T>
static int launch_residual(hipStream_t st, const ResidualArgs& a, int M) {
#define TMX_RESIDUAL(nth, nc)                                                                         \
  if (a.Dp <= 4 * nth * nc) {                                                                         \
    hipLaunchKernelGGL((residual_rows_kernel<T, nth, nc>), dim3(M), dim3(nth), 0, st, a);             \
    return check_launch();                                                                            \
  }
  TMX_RESIDUAL(256, 1)
  TMX_RESIDUAL(512, 1)
  TMX_RESIDUAL(512, 2)
  TMX_RESIDUAL(512, 4)
  TMX_RESIDUAL(512, 8)
#undef TMX_RESIDUAL
  return TMX_ERR_SHAPE;
}

int residual_rows(hipStream_t st, int act, const ResidualArgs& a, int M) {
  if (M <= 0 || a.Dp <= 0 || a.Dp % 64 || a.D > a.Dp || a.D <= 0) return TMX_ERR_SHAPE;
  if (a.y_part && (a.nsplit < 1 || a.nsplit > 4)) return TMX_ERR_ARG;
  if (act == TMX_ACT_BF16) return launch_residual<uint16_t>(st, a, M);
  return act == TMX_ACT_F32 ? launch_residual<float>(st, a, M) : TMX_ERR_ARG;
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

extern "C" int tmx_residual_rows(void* stream, int act, float* x, const void* y, const float* post_w, const float* norm_w,
                                 void* xn, int M, int D, int Dp, float eps, int store) {
  if (!x || !xn) return TMX_ERR_ARG;
  ResidualArgs a = {};
  a.x = x; a.y = y; a.post_w = post_w; a.norm_w = norm_w; a.xn = xn;
  a.D = D; a.Dp = Dp; a.eps = eps; a.store = store;
  return residual_rows((hipStream_t)stream, act, a, M);
}
