// Projections by dense bf16 (or f32) matrices: y = epilogue(x . W^T + bias), optionally one matrix per head.
//
// bf16: the matrices lie in the tile layout of the streamed head (32 rows x 64 columns are 4 KiB in the order the
// lanes of a wave feed them to v_mfma_f32_32x32x16_bf16), so every weight load is 1 KiB of consecutive bytes.
//   up to 128 rows  dense_small_kernel: a weight stream; the waves of a workgroup share 32 (or 2 x 32) output columns
//                   and split K between them, meeting once in LDS, so there are no partial planes in memory and the
//                   epilogue (bias, SwiGLU, sigmoid gate, squared relu) runs on the finished sums
//   more rows       dense_wide_kernel: 256 rows x 32 MT columns per workgroup; the weight slab of a k-step goes
//                   global -> LDS by direct loads, the activations are the B operand straight from memory
// f32: dense_f32_kernel, a plain tiled product on the vector ALU (no matrix pipe, no reduced precision).
#include "tmx_latent_rows.h"

namespace tmx {

__device__ __forceinline__ float silu(float z) { return z / (1.f + expf(-z)); }
__device__ __forceinline__ float sigmoid(float z) { return 1.f / (1.f + expf(-z)); }
__device__ __forceinline__ float relu2(float z) { z = fmaxf(z, 0.f); return z * z; }

// MT: 32-row tiles of x; WK: waves that share K (8 / WK column tiles per workgroup); NT = 2: SwiGLU pairs (a gate
// tile and the up tile N / 64 tiles further).
// XT: x is tiled (act_tile_off): a wave's load is 1 KiB of consecutive bytes instead of 16-byte pieces of 32 rows.
// One workgroup: column tiles bx * 8 / WK .., matrix `head`, slice `slice` of K; lds: kDenseSmallLds bytes.
constexpr int kDenseSmallLds = 65536;
template <int MT, int WK, int NT, bool XT>
__device__ __forceinline__ void dense_small_block(const DenseArgs& a, int bx, int head, int slice, void* lds) {
  constexpr int WN = 8 / WK;
  float* red = reinterpret_cast<float*>(lds);  // [2][8 waves][1024]
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = lane >> 5, nl = lane & 31;
  const int wn = wave / WK, wk = wave % WK;
  const int KT = a.K >> 6;
  const int kts = (KT + a.nsplit - 1) / a.nsplit;
  const int k_beg = slice * kts, k_end = k_beg + kts < KT ? k_beg + kts : KT, klast = k_end - 1;
  const int pair = a.N >> 6;  // tiles from a gate tile to its up tile
  const int tiles = NT == 2 ? pair : a.N >> 5;
  const int tile = bx * WN + wn;
  const int tl = tile < tiles ? tile : tiles - 1;  // waves past the end repeat the last tile (dropped)
  const u32x4_t* wsrc[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n)
    wsrc[n] = reinterpret_cast<const u32x4_t*>(a.w) + ((size_t)head * (a.N >> 5) + tl + n * pair) * KT * 256 + lane;
  const uint16_t* xsrc[MT];
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    if (XT) {
      // (row tiles past the last one repeat it)
      const int mt = m * 32 < a.M ? m : (a.M - 1) >> 5;
      xsrc[m] = reinterpret_cast<const uint16_t*>(a.x) + (size_t)mt * KT * 2048 + lane * 8;
    } else {
      const int row = m * 32 + nl < a.M ? m * 32 + nl : a.M - 1;
      xsrc[m] = reinterpret_cast<const uint16_t*>(a.x) + (size_t)row * a.ldx + head * a.x_head + h * 32;
    }
  }
  f32x16_t acc[NT][MT];
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[n][m][r] = 0.f;

  constexpr int P = MT == 4 ? 1 : 2;  // k-tiles in flight per wave
  u32x4_t wr[P][NT][4], xr[P][MT][4];
  auto load = [&](int kt, auto pc) __attribute__((always_inline)) {
    constexpr int p = decltype(pc)::value;
    kt = kt < klast ? kt : klast;
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
      for (int t = 0; t < 4; ++t) wr[p][n][t] = __builtin_nontemporal_load(wsrc[n] + (size_t)kt * 256 + t * 64);
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int t = 0; t < 4; ++t)
        xr[p][m][t] = *reinterpret_cast<const u32x4_t*>(xsrc[m] + (XT ? (size_t)kt * 2048 + t * 512 : (size_t)kt * 64 + t * 8));
  };
  auto use = [&](auto pc) __attribute__((always_inline)) {
    constexpr int p = decltype(pc)::value;
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
      for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int n = 0; n < NT; ++n)
          acc[n][m] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, xr[p][m][t]),
                                                              __builtin_bit_cast(bf16x8_t, wr[p][n][t]), acc[n][m], 0, 0, 0);
  };
  static_for<P>([&](auto pc) __attribute__((always_inline)) { load(k_beg + wk + decltype(pc)::value * WK, pc); });
  for (int kt = k_beg + wk; kt < k_end; kt += P * WK)
    static_for<P>([&](auto pc) __attribute__((always_inline)) {
      const int k = kt + decltype(pc)::value * WK;
      if (k < k_end) {
        use(pc);
        load(k + P * WK, pc);
      }
    });

  const float b0 = a.bias && slice == 0 ? a.bias[tl * 32 + nl] : 0.f;
  const float b1 = (NT == 2 && a.bias) ? a.bias[(tl + pair) * 32 + nl] : 0.f;
  // Finished bf16 values wait in LDS [rows of x][WN * 32 columns] and leave 8 columns at a time.
  constexpr int OW = WN * 32;
  uint16_t* out_s = reinterpret_cast<uint16_t*>(lds);
  const bool planes = NT == 1 && a.nsplit > 1;
  auto finish = [&](int m, int r, const float* s) __attribute__((always_inline)) {
    const int row = m * 32 + acc_row(r, lane), col = tile * 32 + nl;
    float v = s[0] + b0;
    if (planes) {
      if (row < a.M && tile < tiles) a.y_part[((size_t)slice * a.M + row) * a.N + col] = v;
      return;
    }
    if (NT == 2) v = silu(v) * (s[NT - 1] + b1);
    if (NT == 1 && a.epi == TMX_DENSE_RELU2) v = relu2(v);
    if (a.epi == TMX_DENSE_GATED && row < a.M && tile < tiles)
      v *= sigmoid(bf2f(reinterpret_cast<const uint16_t*>(a.gate)[(size_t)row * a.ldg + head * a.y_head + col]));
    out_s[row * OW + wn * 32 + nl] = f2bf(v);
  };
  constexpr int E = 16 / WK;  // the WK waves of a column tile add their accumulators: each finishes 16 / WK registers
  float s[MT][E][NT];
  if constexpr (WK == 1) {
    static_for<MT * 16>([&](auto ic) __attribute__((always_inline)) {
      constexpr int m = decltype(ic)::value / 16, r = decltype(ic)::value % 16;
#pragma unroll
      for (int n = 0; n < NT; ++n) s[m][r][n] = acc[n][m][r];
    });
  } else {
    static_for<MT * NT>([&](auto ic) __attribute__((always_inline)) {
      constexpr int m = decltype(ic)::value / NT, n = decltype(ic)::value % NT;
      float* buf = red + (decltype(ic)::value & 1) * 8192;
#pragma unroll
      for (int r = 0; r < 16; ++r) buf[wave * 1024 + r * 64 + lane] = acc[n][m][r];
      __syncthreads();  // (the buffer's readers of two rounds ago have passed the last round's barrier)
#pragma unroll
      for (int e = 0; e < E; ++e) {
        float t = 0.f;
#pragma unroll
        for (int w = 0; w < WK; ++w) t += buf[(wn * WK + w) * 1024 + (wk + e * WK) * 64 + lane];
        s[m][e][n] = t;
      }
    });
    if (!planes) __syncthreads();  // every sum is taken: the area is free for the results
  }
  static_for<MT * E>([&](auto ic) __attribute__((always_inline)) {
    constexpr int m = decltype(ic)::value / E, e = decltype(ic)::value % E;
    finish(m, wk + e * WK, s[m][e]);
  });
  if (planes) return;
  __syncthreads();
  const int rows = a.M < MT * 32 ? a.M : MT * 32;
  for (int i = tid; i < rows * (OW / 8); i += 512) {
    const int row = i / (OW / 8), c8 = (i % (OW / 8)) * 8, col = bx * OW + c8;
    if (col >= tiles * 32) continue;
    const int yc = head * a.y_head + col;
    *reinterpret_cast<u32x4_t*>(reinterpret_cast<uint16_t*>(a.y) + (a.y_tiled ? act_tile_off(row, yc, a.ldy) : (size_t)row * a.ldy + yc)) =
        *reinterpret_cast<const u32x4_t*>(out_s + row * OW + c8);
  }
}

template <int MT, int WK, int NT, bool XT>
__global__ __launch_bounds__(512, 2) void dense_small_kernel(DenseArgs a) {
  __shared__ __align__(16) unsigned char lds[kDenseSmallLds];
  dense_small_block<MT, WK, NT, XT>(a, blockIdx.x, blockIdx.y, blockIdx.z, lds);
}

// ---------------------------------------------------------------------------
// More rows: a workgroup of 8 waves multiplies 256 rows of x by MT column tiles (SwiGLU: MT / 2 gate tiles and the
// matching up tiles).  The weight tiles are the A operand and come through a double-buffered LDS slab of TS k-tiles in
// their memory order (a fragment is 1 KiB of consecutive LDS bytes); wave w owns rows 32 w .. 32 w + 31 as the B
// operand, so a lane's accumulator registers are the columns of ONE row, four consecutive ones per store.  LDS reads
// of the next fragment group and the refill of the B registers are pinned between the MFMAs of the current one.
template <int MT, int TS>
struct DenseWide {
  static constexpr size_t LDS = (size_t)2 * MT * TS * 4096;
};

template <int MT, int TS>
__global__ __launch_bounds__(512, 1) void dense_wide_kernel(DenseArgs a, int row_blocks, int col_blocks) {
  // (nsplit > 1: blockIdx.z is the slice of K, of KT / nsplit k-tiles)
  extern __shared__ __align__(16) unsigned char dw_smem[];
  constexpr int kSlab = MT * TS * 4096, kPieces = MT * TS * 4 / 8;  // 1 KiB pieces per wave and step
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = lane >> 5, nl = lane & 31;
  const int cb = (int)blockIdx.x / row_blocks, rb = (int)blockIdx.x % row_blocks;
  if (cb >= col_blocks) return;
  const int head = blockIdx.y;
  const bool swiglu = a.epi == TMX_DENSE_SWIGLU;
  const int KT = a.K >> 6, ntiles = a.N >> 5, pair = a.N >> 6;
  const int row = rb * 256 + wave * 32 + nl, row_l = row < a.M ? row : a.M - 1;
  const int slice = blockIdx.z, nsteps = KT / TS / a.nsplit, first = slice * nsteps, last_step = first + nsteps - 1;
  // column tile of fragment m: MT consecutive ones, or MT / 2 gate tiles and their up tiles
  const int tile0 = swiglu ? cb * (MT / 2) : cb * MT;
  const int live_end = swiglu ? pair : ntiles;
  auto tile_of = [&](int m) {
    const bool up = swiglu && m >= MT / 2;
    const int t = tile0 + (up ? m - MT / 2 : m);
    return (t < live_end ? t : live_end - 1) + (up ? pair : 0);
  };
  const __amdgpu_buffer_rsrc_t rw = make_rsrc(reinterpret_cast<const uint16_t*>(a.w) + (size_t)head * a.N * a.K, (uint32_t)a.N * a.K * 2u);
  const __amdgpu_buffer_rsrc_t rx = make_rsrc(reinterpret_cast<const uint16_t*>(a.x) + head * a.x_head,
                                              ((uint32_t)(a.M - 1) * a.ldx + a.K) * 2u);
  uint32_t wbase[kPieces];
#pragma unroll
  for (int i = 0; i < kPieces; ++i) {
    const int p = wave * kPieces + i;
    wbase[i] = (uint32_t)tile_of(p / (TS * 4)) * KT * 4096u + (p % (TS * 4)) * 1024u;
  }
  const int xv = row_l * a.ldx * 2 + h * 64;

  f32x16_t acc[MT];
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[m][r] = 0.f;
  u32x4_t breg[4 * TS];

  auto load_b = [&](int step, auto gc) __attribute__((always_inline)) {
    constexpr int g = decltype(gc)::value;
    step = step < last_step ? step : last_step;
    breg[g] = __builtin_amdgcn_raw_buffer_load_b128(rx, xv + (g & 3) * 16, (step * TS + (g >> 2)) * 128, 0);
  };
  auto dma_w = [&](int step, int buf) __attribute__((always_inline)) {
    step = step < last_step ? step : last_step;
    unsigned char* base = dw_smem + (size_t)buf * kSlab + wave * kPieces * 1024;
#pragma unroll
    for (int i = 0; i < kPieces; ++i) load_row_to_lds(rw, base + i * 1024, lane * 16, wbase[i] + step * (TS * 4096));
  };
  constexpr int kYounger = 4 * TS;  // B loads requested after the slab's transfers
  auto wait_slab = [&]() __attribute__((always_inline)) {
    __builtin_amdgcn_sched_barrier(0);
    __builtin_amdgcn_s_waitcnt(0x0F70 | (kYounger & 15) | ((kYounger >> 4) << 14));
    __syncthreads();
  };
  auto step_math = [&](int step, int buf) __attribute__((always_inline)) {
    const unsigned char* wb = dw_smem + (size_t)buf * kSlab + lane * 16;
    bf16x8_t wq[2][MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) wq[0][m] = *reinterpret_cast<const bf16x8_t*>(wb + m * TS * 4096);
    __builtin_amdgcn_sched_barrier(0);
    static_for<4 * TS>([&](auto gc) __attribute__((always_inline)) {
      constexpr int g = decltype(gc)::value, cur = g & 1, nxt = cur ^ 1;
      constexpr bool more = g + 1 < 4 * TS;
      const bf16x8_t b = __builtin_bit_cast(bf16x8_t, breg[g]);
      static_for<MT>([&](auto mc) __attribute__((always_inline)) {
        constexpr int m = decltype(mc)::value;
        acc[m] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(wq[cur][m], b, acc[m], 0, 0, 0);
        if constexpr (more) {
          wq[nxt][m] = *reinterpret_cast<const bf16x8_t*>(wb + m * TS * 4096 + (g + 1) * 1024);
          __builtin_amdgcn_sched_barrier(0);
        }
      });
      load_b(step + 1, gc);  // fragment consumed: refill it for the next step
      __builtin_amdgcn_sched_barrier(0);
    });
  };

  dma_w(first, 0);
  static_for<4 * TS>([&](auto gc) __attribute__((always_inline)) { load_b(first, gc); });
  wait_slab();
  for (int step = first; step <= last_step; ++step) {
    const int buf = (step - first) & 1;
    dma_w(step + 1, buf ^ 1);
    __builtin_amdgcn_sched_barrier(0);
    step_math(step, buf);
    wait_slab();
  }
  if (row >= a.M) return;
  uint16_t* yrow = reinterpret_cast<uint16_t*>(a.y) + (size_t)row * a.ldy + head * a.y_head;
  const uint16_t* grow = a.epi == TMX_DENSE_GATED ? reinterpret_cast<const uint16_t*>(a.gate) + (size_t)row * a.ldg + head * a.y_head : nullptr;
  const int F = a.N >> 1;
  auto put = [&](int col, float v0, float v1, float v2, float v3) __attribute__((always_inline)) {
    uint2 w;
    w.x = pack_bf2(v0, v1);
    w.y = pack_bf2(v2, v3);
    *reinterpret_cast<uint2*>(yrow + col) = w;
  };
  if (swiglu) {
    static_for<MT / 2 * 4>([&](auto ic) __attribute__((always_inline)) {
      constexpr int m = decltype(ic)::value / 4, q = decltype(ic)::value % 4;
      const int t = tile0 + m, col = t * 32 + 8 * q + 4 * h;
      if (t >= pair) return;
      float v[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float g = acc[m][4 * q + e] + (a.bias ? a.bias[col + e] : 0.f);
        const float u = acc[m + MT / 2][4 * q + e] + (a.bias ? a.bias[F + col + e] : 0.f);
        v[e] = silu(g) * u;
      }
      put(col, v[0], v[1], v[2], v[3]);
    });
    return;
  }
  static_for<MT * 4>([&](auto ic) __attribute__((always_inline)) {
    constexpr int m = decltype(ic)::value / 4, q = decltype(ic)::value % 4;
    const int t = tile0 + m, col = t * 32 + 8 * q + 4 * h;
    if (t >= ntiles) return;
    float v[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = acc[m][4 * q + e] + (a.bias && slice == 0 ? a.bias[col + e] : 0.f);
    if (a.nsplit > 1) {
      *reinterpret_cast<f32x4_t*>(a.y_part + ((size_t)slice * a.M + row) * a.N + col) = f32x4_t{v[0], v[1], v[2], v[3]};
      return;
    }
    if (a.epi == TMX_DENSE_RELU2) {
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = relu2(v[e]);
    }
    if (grow) {
      const uint2 g = *reinterpret_cast<const uint2*>(grow + col);
      v[0] *= sigmoid(bf_lo(g.x)); v[1] *= sigmoid(bf_hi(g.x));
      v[2] *= sigmoid(bf_lo(g.y)); v[3] *= sigmoid(bf_hi(g.y));
    }
    put(col, v[0], v[1], v[2], v[3]);
  });
}

// ---------------------------------------------------------------------------
// f32: 64 rows x 64 columns per workgroup, 4 x 4 values per thread, K in slices of 16 through LDS.
template <bool SWIGLU>
__global__ __launch_bounds__(256) void dense_f32_kernel(DenseArgs a) {
  constexpr int NT = SWIGLU ? 2 : 1;
  __shared__ __align__(16) float xs[16][68], ws[NT][16][68];
  const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4;
  const int row0 = blockIdx.y * 64, col0 = blockIdx.x * 64, head = blockIdx.z;
  const int cols = SWIGLU ? a.N >> 1 : a.N;
  const float* x = reinterpret_cast<const float*>(a.x) + head * a.x_head;
  const float* w = reinterpret_cast<const float*>(a.w) + (size_t)head * a.N * a.K;
  float acc[NT][4][4] = {};
  const int lr = tid >> 2, lk = (tid & 3) * 4;  // this thread's row (column) and k of a slice transfer
  const float* xp = x + (size_t)(row0 + lr < a.M ? row0 + lr : a.M - 1) * a.ldx + lk;
  const float* wp = w + (size_t)(col0 + lr < cols ? col0 + lr : cols - 1) * a.K + lk;
  for (int k0 = 0; k0 < a.K; k0 += 16) {
    const float4 xv = *reinterpret_cast<const float4*>(xp + k0);
    float4 wv[NT];
#pragma unroll
    for (int n = 0; n < NT; ++n) wv[n] = *reinterpret_cast<const float4*>(wp + (size_t)n * cols * a.K + k0);
    __syncthreads();
    xs[lk][lr] = xv.x; xs[lk + 1][lr] = xv.y; xs[lk + 2][lr] = xv.z; xs[lk + 3][lr] = xv.w;
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      ws[n][lk][lr] = wv[n].x; ws[n][lk + 1][lr] = wv[n].y; ws[n][lk + 2][lr] = wv[n].z; ws[n][lk + 3][lr] = wv[n].w;
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < 16; ++k) {
      float xr[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) xr[i] = xs[k][ty * 4 + i];
#pragma unroll
      for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float wj = ws[n][k][tx * 4 + j];
#pragma unroll
          for (int i = 0; i < 4; ++i) acc[n][i][j] = fmaf(xr[i], wj, acc[n][i][j]);
        }
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int row = row0 + ty * 4 + i, col = col0 + tx * 4 + j;
      if (row >= a.M || col >= cols) continue;
      float v = acc[0][i][j] + (a.bias ? a.bias[col] : 0.f);
      if (SWIGLU) v = silu(v) * (acc[NT - 1][i][j] + (a.bias ? a.bias[cols + col] : 0.f));
      if (a.epi == TMX_DENSE_RELU2) v = relu2(v);
      if (a.epi == TMX_DENSE_GATED)
        v *= sigmoid(reinterpret_cast<const float*>(a.gate)[(size_t)row * a.ldg + head * a.y_head + col]);
      reinterpret_cast<float*>(a.y)[(size_t)row * a.ldy + head * a.y_head + col] = v;
    }
}

// ---------------------------------------------------------------------------
template <int MT, int WK, int NT, bool XT>
static int launch_small(hipStream_t st, const DenseArgs& a) {
  const int tiles = NT == 2 ? a.N / 64 : a.N / 32, wn = 8 / WK;
  hipLaunchKernelGGL((dense_small_kernel<MT, WK, NT, XT>), dim3((tiles + wn - 1) / wn, a.heads, a.nsplit), dim3(512), 0, st, a);
  return check_launch();
}
// Queries into the latent space (one matrix per head) and the row part of latent attention, in one launch: the first
// gx * heads workgroups are the projection's, the others one row each.
template <int MT, int WK>
__global__ __launch_bounds__(512, 2) void latent_q_rows_kernel(DenseArgs a, LatentRowsArgs r, int gx) {
  __shared__ __align__(16) unsigned char lds[kDenseSmallLds];
  const int b = blockIdx.x, nq = gx * a.heads;
  if (b < nq) dense_small_block<MT, WK, 1, false>(a, b % gx, b / gx, 0, lds);
  else latent_rows_block<uint16_t, 512>(r, b - nq, reinterpret_cast<float*>(lds));
}
template <int MT>
static int launch_q_rows(hipStream_t st, const DenseArgs& a, const LatentRowsArgs& r) {
  const int wk = a.K >= 128 ? 2 : 1, wn = 8 / wk, gx = (a.N / 32 + wn - 1) / wn;
  const dim3 grid(gx * a.heads + a.M);
  if (wk == 2) hipLaunchKernelGGL((latent_q_rows_kernel<MT, 2>), grid, dim3(512), 0, st, a, r, gx);
  else hipLaunchKernelGGL((latent_q_rows_kernel<MT, 1>), grid, dim3(512), 0, st, a, r, gx);
  return check_launch();
}
int latent_q_rows(hipStream_t st, DenseArgs a, const LatentRowsArgs& r) {
  if (a.M <= 0 || a.M > 128 || a.K % 64 || a.N % 32 || a.heads <= 0 || a.bias || a.epi != TMX_DENSE_PLAIN || a.x_tiled || a.y_tiled ||
      a.ldx % 8 || a.x_head % 8 || a.ldy % 8 || a.y_head % 8 || r.rot <= 0 || r.rot % 2 || r.rot > r.rot_p || r.rank <= 0 ||
      r.rank > r.rank_p || !latent_attn_ok(r.rank_p, r.rot_p))
    return TMX_ERR_SHAPE;
  a.nsplit = 1;
  if (a.M <= 32) return launch_q_rows<1>(st, a, r);
  if (a.M <= 64) return launch_q_rows<2>(st, a, r);
  return launch_q_rows<4>(st, a, r);
}

template <int MT, int NT, bool XT>
static int launch_small_k(hipStream_t st, const DenseArgs& a) {
  const int KT = (a.K >> 6) / a.nsplit;
  if (KT >= 8) return launch_small<MT, 8, NT, XT>(st, a);
  if (KT >= 4) return launch_small<MT, 4, NT, XT>(st, a);
  if (KT >= 2) return launch_small<MT, 2, NT, XT>(st, a);
  return launch_small<MT, 1, NT, XT>(st, a);
}
template <int MT, int NT>
static int launch_small_x(hipStream_t st, const DenseArgs& a) {
  return a.x_tiled ? launch_small_k<MT, NT, true>(st, a) : launch_small_k<MT, NT, false>(st, a);
}

int dense_num_splits(int act, int M, int K, int N) {
  if (act != TMX_ACT_BF16) return 1;
  const int KT = K >> 6, cus = device_cus();
  int ns = 1;
  if (M <= 128) {
    // two workgroups per CU, at least two k-tiles per wave
    while (ns < 4 && (N / 32) * ns * 2 <= 2 * cus && KT / (2 * ns) >= 16) ns *= 2;
    return ns;
  }
  // 256 x 256 blocks while they do not fill the CUs
  const long wgs = (long)((M + 255) / 256) * ((N + 255) / 256);
  while (ns < 4 && wgs * ns * 2 <= cus && KT % (4 * ns) == 0 && KT / (2 * ns) >= 8) ns *= 2;
  return ns;
}

template <int MT, int TS>
static int launch_wide(hipStream_t st, const DenseArgs& a) {
  static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(&dense_wide_kernel<MT, TS>),
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, (int)DenseWide<MT, TS>::LDS);
  if (attr != hipSuccess) return TMX_ERR_LAUNCH;
  const int per = a.epi == TMX_DENSE_SWIGLU ? MT / 2 : MT, tiles = a.epi == TMX_DENSE_SWIGLU ? a.N / 64 : a.N / 32;
  const int rb = (a.M + 255) / 256, cb = (tiles + per - 1) / per;
  hipLaunchKernelGGL((dense_wide_kernel<MT, TS>), dim3(rb * cb, a.heads, a.nsplit), dim3(512), (DenseWide<MT, TS>::LDS), st, a, rb, cb);
  return check_launch();
}

int dense_linear(hipStream_t st, int act, const DenseArgs& args) {
  DenseArgs a = args;
  if (a.nsplit < 1) a.nsplit = 1;
  const bool swiglu = a.epi == TMX_DENSE_SWIGLU;
  if (a.M <= 0 || a.K <= 0 || a.N <= 0 || a.heads <= 0 || a.heads > 65535 || a.K % 64 || a.N % 32) return TMX_ERR_SHAPE;
  if (swiglu && (a.N % 64 || a.heads != 1)) return TMX_ERR_SHAPE;
  if (a.heads != 1 && a.bias) return TMX_ERR_ARG;
  if (a.nsplit > 1 && (!a.y_part || a.heads != 1 || a.epi != TMX_DENSE_PLAIN || act != TMX_ACT_BF16)) return TMX_ERR_ARG;
  if ((a.x_tiled || a.y_tiled) && (act != TMX_ACT_BF16 || a.M > 128 || (a.x_tiled && a.heads != 1) || (a.y_tiled && a.ldy % 64)))
    return TMX_ERR_ARG;
  if (act == TMX_ACT_F32) {
    if (a.ldx % 4 || a.x_head % 4) return TMX_ERR_SHAPE;
    const int cols = swiglu ? a.N / 2 : a.N;
    const dim3 grid((cols + 63) / 64, (a.M + 63) / 64, a.heads);
    if (swiglu) hipLaunchKernelGGL(dense_f32_kernel<true>, grid, dim3(256), 0, st, a);
    else hipLaunchKernelGGL(dense_f32_kernel<false>, grid, dim3(256), 0, st, a);
    return check_launch();
  }
  if (act != TMX_ACT_BF16) return TMX_ERR_ARG;
  if (a.ldx % 8 || a.x_head % 8 || a.ldy % 8 || a.y_head % 8 || a.ldg % 4) return TMX_ERR_SHAPE;
  if (a.M <= 128) {
    if (swiglu) {
      if (a.M <= 32) return launch_small_x<1, 2>(st, a);
      if (a.M <= 64) return launch_small_x<2, 2>(st, a);
      return launch_small_x<4, 2>(st, a);
    }
    if (a.M <= 32) return launch_small_x<1, 1>(st, a);
    if (a.M <= 64) return launch_small_x<2, 1>(st, a);
    return launch_small_x<4, 1>(st, a);
  }
  // buffer descriptors hold byte offsets of 31 bits
  if ((size_t)a.N * a.K * 2 >= (1u << 31) || (size_t)a.M * a.ldx * 2 >= (1u << 31)) return TMX_ERR_SHAPE;
  const int tiles = swiglu ? a.N / 64 : a.N / 32, per8 = swiglu ? 4 : 8;
  const long wgs = (long)((a.M + 255) / 256) * ((tiles + per8 - 1) / per8) * a.heads * a.nsplit;
  const bool wide8 = wgs >= device_cus() && tiles > per8 / 2;
  if ((a.K >> 6) % (2 * a.nsplit) == 0) return wide8 ? launch_wide<8, 2>(st, a) : launch_wide<4, 2>(st, a);
  if ((a.K >> 6) % a.nsplit) return TMX_ERR_SHAPE;
  return wide8 ? launch_wide<8, 1>(st, a) : launch_wide<4, 1>(st, a);
}

}  // namespace tmx

using namespace tmx;

extern "C" int tmx_dense_linear(void* stream, int act, const void* x, int ldx, int x_head, const void* w,
                                const float* bias, const void* gate, int ldg, void* y, int ldy, int y_head, int M,
                                int K, int N, int heads, int epilogue) {
  if (!x || !w || !y || (epilogue == TMX_DENSE_GATED && !gate)) return TMX_ERR_ARG;
  if (epilogue < TMX_DENSE_PLAIN || epilogue > TMX_DENSE_RELU2) return TMX_ERR_UNSUPPORTED;
  DenseArgs a = {};
  a.x = x; a.ldx = ldx; a.x_head = x_head;
  a.w = w; a.bias = bias; a.gate = gate; a.ldg = ldg;
  a.y = y; a.ldy = ldy; a.y_head = y_head;
  a.M = M; a.K = K; a.N = N; a.heads = heads; a.epi = epilogue;
  return dense_linear((hipStream_t)stream, act, a);
}
