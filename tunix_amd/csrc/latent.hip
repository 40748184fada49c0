// Latent attention: every token caches one latent vector c (normed) and one rotated key part shared by all heads;
// a head's keys and values are linear in c, so its query is moved into the latent space (q~ = W_uk^T q, a batched
// projection) and the attention runs on the cache rows themselves:
//   score_j = (q~ . c_j + rot(q_r) . rot(k_r)_j) scale,   out~ = sum_j p_j c_j,   value = W_uv out~
// All heads read the same row, once: keys are its rank_p + rot_p columns, values its first rank_p.
//
//   latent_rows_kernel    rotation of the queries, norm + rotation of the new cache row
//   latent_attn_kernel    the walk over the cache on the matrix pipe (one or many tokens per sequence)
//   latent_combine_kernel merge of the splits of a query row
//   latent_attn_f32_kernel the same attention in f32 on the vector ALU
#include "tmx_latent_rows.h"

namespace tmx {

template <typename T>
__global__ __launch_bounds__(256) void latent_rows_kernel(LatentRowsArgs a) {
  __shared__ float smem[4];
  latent_rows_block<T, 256>(a, blockIdx.x, smem);
}

// ---------------------------------------------------------------------------
// The walk.  Query rows of a sequence are its (token, head) pairs, 32 of them the columns of an MFMA tile: as in the
// grouped-query kernels, scores^T [position, query] = rows . Q^T and out^T [column, query] += rows^T . P^T, with a
// lane owning one query.  A block of 32 cache rows goes global -> LDS once (direct loads, 16-byte chunks XOR-swizzled
// by row) and serves both products: as the A operand of the scores by rows, and transposed (ds_read_b64_tr_b16) as
// the A operand of the output.  Probabilities enter the product as bf16 hi + lo.
// The four waves of a workgroup are WQ groups of query rows x WP groups of positions x WC groups of output columns:
//   SHARED (many query rows per sequence): WP = 1, all waves walk the same blocks;
//   else (up to 32 query rows): WQ = 1, the position groups take different blocks and meet through LDS at the end.
// WC = 2 at the full latent width, where the accumulators of 32 queries and the query fragments of one wave would not
// fit its registers: two waves share the query rows, each with half of the output columns.
//   PAIR (SHARED with WC = 2): a round takes two blocks; each wave of a pair scores one of them and hands its
//   probabilities to the other through LDS, so no score is computed twice.
//   else with WC = 2: both waves make the scores.
// KVT: latent width / 32, RT: width of the rotated part / 64.
template <int KVT, int RT, bool SHARED>
struct LatentShape {
  static constexpr int WC = KVT > 8 ? 2 : 1, WQ = SHARED ? 4 / WC : 1, WP = SHARED ? 1 : 4 / WC;
  static constexpr bool PAIR = SHARED && WC == 2;
  static constexpr int kLd = KVT * 32 + RT * 64;
  static constexpr size_t kTile = (size_t)32 * kLd * 2;
  static constexpr int kGroup = PAIR ? 2 : 1;                     // tiles of a position group and round
  static constexpr size_t kExchange = PAIR ? 4 * 4096 : 0;        // probabilities of a wave's block
  static constexpr int kBufs = 2 * WP * kGroup * kTile + kExchange <= 160 * 1024 ? 2 : 1;
  static constexpr size_t kTiles = kBufs * WP * kGroup * kTile;
  static constexpr size_t kMerge = SHARED ? 0 : (size_t)(WP / 2) * (KVT * 16 * 64 * 4 + WC * 2 * 32 * 4);
  static constexpr size_t kBytes = kTiles + kExchange > kMerge ? kTiles + kExchange : kMerge;
};

// 16-byte chunk c of row r lies at chunk c ^ swz(r).  Rows whose stride is a multiple of the 64 banks are told apart
// by four bits of the row; rows of an odd number of 128 bytes already alternate between the two halves of the banks
// and take three.  Row bits 0, 1 (1) go to the high bits so that the four rows of a transposing read differ by
// whole groups of four chunks.
template <int CPR>
__device__ __forceinline__ constexpr int latent_swz(int row) {
  return CPR % 16 == 0 ? ((row & 3) << 2) | ((row >> 2) & 3) : (((row >> 1) & 1) << 2) | ((row >> 2) & 3);
}

template <int KVT, int RT, bool SHARED>
__global__ __launch_bounds__(256, 1) void latent_attn_kernel(LatentAttnArgs a) {
  using SH = LatentShape<KVT, RT, SHARED>;
  extern __shared__ __align__(16) unsigned char la_smem[];
  constexpr int LD = SH::kLd, CPR = LD / 8, KS = LD / 16, CP = KVT * 32;
  constexpr int WC = SH::WC, WP = SH::WP, KC = KVT / WC;  // KC: column tiles of a wave
  constexpr bool PAIR = SH::PAIR;
  constexpr int kTile = 32 * LD;                          // elements
  constexpr int WPW = 4 / WP;                             // waves per position group
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int h = lane >> 5, qi = lane & 31;
  const int wc = wave % WC, wq = SHARED ? wave / WC : 0, wp = SHARED ? 0 : wave / WC;
  const int wg = wave % WPW;  // wave within its position group
  const int seq = blockIdx.y, split = blockIdx.z;
  const int rows = a.tpp * a.H;  // query rows of a sequence
  const int q0 = blockIdx.x * (32 * SH::WQ);
  const int qr = q0 + wq * 32 + qi, qr_l = qr < rows ? qr : rows - 1;
  const size_t qrow = (size_t)seq * rows + qr_l;

  const __amdgpu_buffer_rsrc_t rc = make_rsrc(reinterpret_cast<const uint16_t*>(a.cache) + (size_t)seq * a.C * LD,
                                              (uint32_t)a.C * LD * 2u);  // rows past the cache read zero
  uint16_t* tiles = reinterpret_cast<uint16_t*>(la_smem) + wp * SH::kBufs * SH::kGroup * kTile;
  // 32 rows of LD columns into a tile, 1 KiB per load, shared by n waves of which this is number i0: load i0 + n i, whose
  // byte offset in the 32 rows is this lane's row_off(i0 + n i)
  auto row_off = [&](int ld) {
    const int g = ld * 64 + lane, row = g / CPR, slot = g - row * CPR;
    return (row * CPR + (slot ^ latent_swz<CPR>(row))) * 16;
  };
  constexpr int kDma = CPR / 2 / WPW;  // loads of a wave per tile
  int doff[kDma];
#pragma unroll
  for (int i = 0; i < kDma; ++i) doff[i] = row_off(wg + WPW * i);
  auto dma = [&](int row0, uint16_t* tile) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < kDma; ++i) load_row_to_lds(rc, tile + (wg + WPW * i) * 512, doff[i], row0 * (LD * 2));
  };
  const uint8_t* mrow = a.input_mask + (size_t)seq * a.buf_len;
  auto mask_byte = [&](int blk) __attribute__((always_inline)) {
    const int p = blk * 32 + qi;
    return (h == 0 && p < a.buf_len) ? mrow[p] : (uint8_t)0;
  };

  f32x16_t o[KC];
#pragma unroll
  for (int c = 0; c < KC; ++c)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[c][r] = 0.f;
  // running maximum and sum of the softmax; exponentials are powers of two throughout (scores times log2 e), a masked
  // score is far below the maximum of a row that has seen none
  constexpr float kLog2e = 1.44269504f, kUnseen = -1e30f, kHidden = -2e30f;
  const float scale2 = a.scale * kLog2e;
  float m = kUnseen, l = 0.f;

  // Blocks are dealt out in turn to the position groups of all splits: the first one does not depend on *step, so its
  // transfer starts at once.  All groups of a workgroup run the same number of rounds.
  constexpr int BG = PAIR ? 2 : WP;  // blocks of a workgroup and round
  const int blk0 = split * BG + (PAIR ? wc : wp), stride = a.nsplit * BG;
  auto blk_of = [&](int round) { return blk0 + round * stride; };  // the block this wave scores
  auto fetch = [&](int round, int buf) __attribute__((always_inline)) {
    if constexpr (PAIR) {  // (both tiles also where the second block lies behind the last: zeros or older rows)
#pragma unroll
      for (int e = 0; e < 2; ++e) dma((split * BG + e + round * stride) * 32, tiles + (buf * 2 + e) * kTile);
    } else {
      dma(blk_of(round) * 32, tiles + buf * kTile);
    }
  };
  constexpr int kBuf0 = PAIR && SH::kBufs == 2 ? 1 : 0;  // tile buffer of round 0
  // The query fragments come through LDS as well (read from memory they would be 16-byte pieces of 32 rows per load):
  // the query groups of the workgroup, two at a time, through the tiles that are not in use yet.
  u32x4_t qf[KS];
  {
    // the first tiles start with the queries where there is room beside them: they go to the buffer that round 0 uses
    constexpr bool early = (!SHARED || PAIR) && SH::kBufs == 2;
    const __amdgpu_buffer_rsrc_t rq = make_rsrc(reinterpret_cast<const uint16_t*>(a.q) + (size_t)seq * rows * LD, (uint32_t)rows * LD * 2u);
    uint16_t* const lds = reinterpret_cast<uint16_t*>(la_smem);
    if (early) fetch(0, kBuf0);
    constexpr int kStage = SHARED ? 2 : 1;             // query groups per turn
    constexpr int kQTile = early && !PAIR ? 1 : 0;    // tile (of the workgroup) they pass through
#pragma unroll
    for (int g = 0; g < SH::WQ; g += kStage) {
#pragma unroll
      for (int e = 0; e < kStage; ++e)
#pragma unroll
        for (int i = 0; i < CPR / 8; ++i)
          load_row_to_lds(rq, lds + (kQTile + e) * kTile + (wave + 4 * i) * 512, row_off(wave + 4 * i), (q0 + (g + e) * 32) * (LD * 2));
      __builtin_amdgcn_s_waitcnt(0x0F70);
      __syncthreads();
      if (wq >= g && wq < g + kStage) {
        const uint16_t* qb = lds + (kQTile + wq - g) * kTile + qi * LD;
#pragma unroll
        for (int t = 0; t < KS; ++t)
          qf[t] = *reinterpret_cast<const u32x4_t*>(qb + (((KS * h + t) ^ latent_swz<CPR>(qi)) << 3));
      }
      __syncthreads();
    }
    if (!early && SH::kBufs == 2) fetch(0, kBuf0);
  }
  const int step0 = max(min(*a.step, min(a.C, a.buf_len) - a.tpp), 0);  // clamped: every slot read lies in the cache
  const int limit = step0 + qr_l / a.H;                               // newest slot this query sees
  const int limit0 = step0 + min(q0 + wq * 32, rows - 1) / a.H;       // the smallest one in the wave
  const int b_end = (step0 + (min(q0 + 32 * SH::WQ, rows) - 1) / a.H + 32) >> 5;  // blocks up to the workgroup's newest slot
  const int rounds = b_end > split * BG ? (b_end - split * BG + stride - 1) / stride : 0;
  uint8_t mb = mask_byte(blk_of(0));
  // transposed fragments of the output product: lane (column 32 c + qi, h) takes two runs of four consecutive rows
  // (see gqa_tile_walk)
  const int k4 = (lane & 15) >> 2, q4 = lane & 3, g2 = (lane >> 4) & 1;
  const uint32_t lsw = ((2 * g2 + (q4 >> 1)) ^ latent_swz<CPR>(4 * h + k4)) * 16;
  const uint32_t vbase = ((4 * h + k4) * LD + 4 * (q4 & 1) + wc * KC * 32) * 2;
  const int kbase = qi * LD;
  constexpr int R = 4;  // LDS fragments in flight
  auto lds_addr = [](const uint16_t* p) __attribute__((always_inline)) {
    return (uint32_t)(uintptr_t)(__attribute__((address_space(3))) const uint16_t*)p;
  };
  // scaled scores of a block; the largest one of this lane's query in mn
  auto scores = [&](const uint16_t* kt, int blk, uint32_t mbits, f32x16_t& sacc, float& mn) __attribute__((always_inline)) {
    const int sw = latent_swz<CPR>(qi);
    bf16x8_t kf[R];
    auto load_k = [&](auto tc) __attribute__((always_inline)) {
      constexpr int t = decltype(tc)::value;
      kf[t % R] = *reinterpret_cast<const bf16x8_t*>(kt + kbase + (((KS * h + t) ^ sw) << 3));
    };
#pragma unroll
    for (int r = 0; r < 16; ++r) sacc[r] = 0.f;
    static_for<R>([&](auto tc) __attribute__((always_inline)) { load_k(tc); });
    __builtin_amdgcn_sched_barrier(0);
    static_for<KS>([&](auto tc) __attribute__((always_inline)) {  // lane (position, h) multiplies the half h of its row
      constexpr int t = decltype(tc)::value;
      sacc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf[t % R], __builtin_bit_cast(bf16x8_t, qf[t]), sacc, 0, 0, 0);
      if constexpr (t + R < KS) load_k(IC<t + R>{});
      __builtin_amdgcn_sched_barrier(0);
    });
    mn = kUnseen;
    if (mbits == 0xFFFFFFFFu && blk * 32 + 31 <= limit0) {  // every query of the wave sees the whole block
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        sacc[r] *= scale2;
        mn = fmaxf(mn, sacc[r]);
      }
    } else {
      const int lim = limit - blk * 32 - 4 * h;
      const uint32_t mb2 = mbits >> (4 * h);
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int pc = (r >> 2) * 8 + (r & 3);  // acc_row(r, lane) without the lane's half
        sacc[r] = pc <= lim && ((mb2 >> pc) & 1u) ? sacc[r] * scale2 : kHidden;
        mn = fmaxf(mn, sacc[r]);
      }
    }
    mn = fmaxf(mn, __shfl_xor(mn, 32, 64));
  };
  // The reference point of the exponentials moves only when a score has left it by more than 12: until then the
  // probabilities stay below 2^12 and the accumulators need no rescaling.
  auto move_reference = [&](float mn) __attribute__((always_inline)) {
    if (__any(mn > m + 12.f)) {
      mn = fmaxf(mn, m);
      const float alpha = __builtin_amdgcn_exp2f(m - mn);
      m = mn;
      l *= alpha;
#pragma unroll
      for (int c = 0; c < KC; ++c)
#pragma unroll
        for (int r = 0; r < 16; ++r) o[c][r] *= alpha;
    }
  };
  // probabilities as bf16 hi (p[0], p[1]) and lo (p[2], p[3]), 16 positions each
  auto probabilities = [&](const f32x16_t& sacc, u32x4_t* p) __attribute__((always_inline)) {
#pragma unroll
    for (int r = 0; r < 16; r += 2) {
      const float p0 = __builtin_amdgcn_exp2f(sacc[r] - m), p1 = __builtin_amdgcn_exp2f(sacc[r + 1] - m);
      const uint32_t hi = pack_bf2(p0, p1);
      p[r >> 3][(r >> 1) & 3] = hi;
      p[2 + (r >> 3)][(r >> 1) & 3] = pack_bf2(p0 - bf_lo(hi), p1 - bf_hi(hi));
      l += p0 + p1;
    }
  };
  // Transposed fragments f = (half kb2 of the block, column tile c) of a tile.  (The reads are spelled in assembly: for
  // the builtin the compiler waits for every direct-to-LDS load in flight, i.e. for the next tile; the waits in
  // `product` count them instead.)
  u32x2_t vf[R][2];
  auto load_v = [&](uint32_t vb, auto fc) __attribute__((always_inline)) {
    constexpr int f = decltype(fc)::value, kb2 = f / KC, c = f % KC;
    static_for<2>([&](auto ac) __attribute__((always_inline)) {
      constexpr int a2 = decltype(ac)::value, row0 = 16 * kb2 + 8 * a2;
      const uint32_t ad = vb + (lsw ^ (uint32_t)(((4 * c) ^ latent_swz<CPR>(row0)) * 16));
      u32x2_t& dst = vf[f % R][a2];
      asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(dst) : "v"(ad), "i"(row0 * LD * 2));
    });
  };
  auto request_v = [&](const uint16_t* kt) __attribute__((always_inline)) {  // the first R fragments of a tile
    const uint32_t vb = lds_addr(kt) + vbase;
    static_for<R>([&](auto fc) __attribute__((always_inline)) { load_v(vb, fc); });
    __builtin_amdgcn_sched_barrier(0);
  };
  // out^T += rows^T . P^T, 16 positions (accumulator registers 8 kb2 .. 8 kb2 + 7) per MFMA
  auto product = [&](const uint16_t* kt, const u32x4_t* p) __attribute__((always_inline)) {
    const uint32_t vb = lds_addr(kt) + vbase;
    static_for<2 * KC>([&](auto fc) __attribute__((always_inline)) {
      constexpr int f = decltype(fc)::value, kb2 = f / KC, c = f % KC;
      constexpr int kLater = 2 * KC - 1 - f < R - 1 ? 2 * KC - 1 - f : R - 1;  // fragments requested behind this one
      u32x2_t &v0 = vf[f % R][0], &v1 = vf[f % R][1];
      asm volatile("s_waitcnt lgkmcnt(%2)" : "+v"(v0), "+v"(v1) : "i"(2 * kLater));
      const u32x4_t v = {v0.x, v0.y, v1.x, v1.y};
      o[c] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, v), __builtin_bit_cast(bf16x8_t, p[kb2]),
                                                     o[c], 0, 0, 0);
      o[c] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, v),
                                                     __builtin_bit_cast(bf16x8_t, p[2 + kb2]), o[c], 0, 0, 0);
      if constexpr (f + R < 2 * KC) load_v(vb, IC<f + R>{});
      __builtin_amdgcn_sched_barrier(0);
    });
  };
  // LDS traffic between the waves of a pair, past the transfers in flight: a barrier that waits for LDS operations only
  auto lds_barrier = [&]() __attribute__((always_inline)) {
    asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
  };
  const uint32_t xch = lds_addr(reinterpret_cast<const uint16_t*>(la_smem)) + (uint32_t)SH::kTiles;
  const uint32_t own_x = xch + wave * 4096 + lane * 16, mate_x = xch + (wave ^ 1) * 4096 + lane * 16;

  for (int round = 0; round < rounds; ++round) {
    const int buf = SH::kBufs == 2 ? (round & 1) ^ kBuf0 : 0;
    if (SH::kBufs == 1) {
      __syncthreads();  // the last round's reads are complete
      if (PAIR || blk_of(round) < b_end) fetch(round, 0);
    }
    const uint32_t mbits = (uint32_t)__ballot(mb != 0);
    __builtin_amdgcn_s_waitcnt(0x0F70);  // this round's tiles have landed
    __syncthreads();
    mb = mask_byte(blk_of(round + 1));
    if (SH::kBufs == 2 && (PAIR ? round + 1 < rounds : blk_of(round + 1) < b_end)) fetch(round + 1, buf ^ 1);
    if constexpr (PAIR) {
      const uint16_t *own = tiles + (buf * 2 + wc) * kTile, *mate = tiles + (buf * 2 + (wc ^ 1)) * kTile;
      f32x16_t sacc;
      float mn, mn2;
      u32x4_t p[4], p2[4];
      scores(own, blk_of(round), mbits, sacc, mn);
      // the pair agrees on the reference point: a wave leaves its maximum in the mate's exchange area, which only the
      // mate writes to afterwards
      asm volatile("ds_write_b32 %0, %1" ::"v"(mate_x), "v"(mn) : "memory");
      lds_barrier();
      asm volatile("ds_read_b32 %0, %1\n\ts_waitcnt lgkmcnt(0)" : "=v"(mn2) : "v"(own_x) : "memory");
      request_v(own);
      move_reference(fmaxf(mn, mn2));
      probabilities(sacc, p);
      static_for<4>([&](auto ic) __attribute__((always_inline)) {
        constexpr int i = decltype(ic)::value;
        const u32x4_t& src = p[i];
        const uint32_t at = own_x;
        asm volatile("ds_write_b128 %0, %1 offset:%2" ::"v"(at), "v"(src), "i"(i * 1024) : "memory");
      });
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
      product(own, p);
      lds_barrier();
      static_for<4>([&](auto ic) __attribute__((always_inline)) {
        constexpr int i = decltype(ic)::value;
        u32x4_t& dst = p2[i];
        const uint32_t at = mate_x;
        asm volatile("ds_read_b128 %0, %1 offset:%2" : "=v"(dst) : "v"(at), "i"(i * 1024) : "memory");
      });
      request_v(mate);
      {
        u32x4_t &q0_ = p2[0], &q1_ = p2[1], &q2_ = p2[2], &q3_ = p2[3];
        asm volatile("s_waitcnt lgkmcnt(%4)" : "+v"(q0_), "+v"(q1_), "+v"(q2_), "+v"(q3_) : "i"(2 * R));
      }
      product(mate, p2);
    } else if (blk_of(round) < b_end) {
      const uint16_t* kt = tiles + buf * kTile;
      f32x16_t sacc;
      float mn;
      u32x4_t p[4];
      scores(kt, blk_of(round), mbits, sacc, mn);
      request_v(kt);  // they do not wait for the softmax
      move_reference(mn);
      probabilities(sacc, p);
      product(kt, p);
    }
  }
  if constexpr (PAIR) {  // each wave has counted its own blocks
    float l2;
    lds_barrier();
    asm volatile("ds_write_b32 %0, %1" ::"v"(mate_x), "v"(l) : "memory");
    lds_barrier();
    asm volatile("ds_read_b32 %0, %1\n\ts_waitcnt lgkmcnt(0)" : "=v"(l2) : "v"(own_x) : "memory");
    l += l2;
  }
  l += __shfl_xor(l, 32, 64);
  if constexpr (WP > 1) {
    // merge the position groups: the upper half of them hands its state to the lower half, until one is left
    constexpr int kPart = KVT * 16 * 64;
    float* mf = reinterpret_cast<float*>(la_smem);
    float* ml = mf + (WP / 2) * kPart;  // [slot][column group][m, l][32]
    auto put = [&](int s) __attribute__((always_inline)) {
#pragma unroll
      for (int c = 0; c < KC; ++c)
#pragma unroll
        for (int r = 0; r < 16; ++r) mf[s * kPart + (((wc * KC + c) * 16 + r) << 6) + lane] = o[c][r];
      if (h == 0) {
        ml[(s * WC + wc) * 64 + qi] = m;
        ml[(s * WC + wc) * 64 + 32 + qi] = l;
      }
    };
    auto take = [&](int s) __attribute__((always_inline)) {
      const float m2 = ml[(s * WC + wc) * 64 + qi], l2 = ml[(s * WC + wc) * 64 + 32 + qi];
      const float mm = fmaxf(m, m2), w1 = __builtin_amdgcn_exp2f(m - mm), w2 = __builtin_amdgcn_exp2f(m2 - mm);
#pragma unroll
      for (int c = 0; c < KC; ++c)
#pragma unroll
        for (int r = 0; r < 16; ++r)
          o[c][r] = o[c][r] * w1 + mf[s * kPart + (((wc * KC + c) * 16 + r) << 6) + lane] * w2;
      l = l * w1 + l2 * w2;
      m = mm;
    };
#pragma unroll
    for (int n = WP / 2; n > 0; n >>= 1) {
      __syncthreads();
      if (wp >= n && wp < 2 * n) put(wp - n);
      __syncthreads();
      if (wp < n) take(wp);
    }
    if (wp != 0) return;
  }
  constexpr int kOut = KC * 32 + 8;  // PAIR: row stride of the results in LDS
  if constexpr (PAIR) __syncthreads();  // the tiles are free
  if ((PAIR && a.nsplit == 1 ? q0 + wq * 32 : qr) >= rows) return;
  if (a.nsplit == 1) {
    float w = 1.f;
    if (a.sink) {  // one more term of the denominator, without a value
      const float s = a.sink[qr % a.H] * kLog2e, mm = fmaxf(m, s);
      w = __builtin_amdgcn_exp2f(m - mm);
      l = l * w + __builtin_amdgcn_exp2f(s - mm);
    }
    const float inv = l > 0.f ? w / l : 0.f;
    uint16_t* dst = reinterpret_cast<uint16_t*>(a.out) + qrow * CP + wc * KC * 32;
    if constexpr (PAIR) dst = reinterpret_cast<uint16_t*>(la_smem) + wave * kOut * 32 + qi * kOut;
#pragma unroll
    for (int c = 0; c < KC; ++c)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        uint2 v;
        v.x = pack_bf2(o[c][4 * i] * inv, o[c][4 * i + 1] * inv);
        v.y = pack_bf2(o[c][4 * i + 2] * inv, o[c][4 * i + 3] * inv);
        *reinterpret_cast<uint2*>(dst + 32 * c + 8 * i + 4 * h) = v;
      }
    if constexpr (PAIR) {  // the wave's own rows, out again in whole lines
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
      constexpr int CPO = KC * 4;  // 16-byte chunks of a row
#pragma unroll
      for (int i = 0; i < 32 * CPO / 64; ++i) {
        const int g = i * 64 + lane, row = g / CPO, ch = g % CPO, q = q0 + wq * 32 + row;
        const u32x4_t v = *reinterpret_cast<const u32x4_t*>(reinterpret_cast<const uint16_t*>(la_smem) + wave * kOut * 32 + row * kOut + ch * 8);
        if (q < rows)
          *reinterpret_cast<u32x4_t*>(reinterpret_cast<uint16_t*>(a.out) + ((size_t)seq * rows + q) * CP + wc * KC * 32 + ch * 8) = v;
      }
    }
    return;
  }
  float* pr = a.partial + (qrow * a.nsplit + split) * (CP + 4);
#pragma unroll
  for (int c = 0; c < KC; ++c)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      float* d = pr + 32 * (wc * KC + c) + 8 * i + 4 * h;
      *reinterpret_cast<f32x4_t*>(d) = f32x4_t{o[c][4 * i], o[c][4 * i + 1], o[c][4 * i + 2], o[c][4 * i + 3]};
    }
  if (h == 0 && wc == 0) {
    pr[CP] = m * (1.f / kLog2e);  // (natural units, as the sink)
    pr[CP + 1] = l;
  }
}

// One workgroup per query row: the softmax-weighted sum of its splits, then the sink.
__global__ __launch_bounds__(256) void latent_combine_kernel(LatentAttnArgs a) {
  const int CP = a.rank_p;
  const size_t row = blockIdx.x;
  const float* pr = a.partial + row * a.nsplit * (CP + 4);  // [split][CP values | max | sum | -]
  float mm = a.sink ? a.sink[row % a.H] : -1e30f;
  const float sink = mm;
  for (int s = 0; s < a.nsplit; ++s) mm = fmaxf(mm, pr[(size_t)s * (CP + 4) + CP]);
  float l = a.sink ? __expf(sink - mm) : 0.f;
  for (int s = 0; s < a.nsplit; ++s) l += pr[(size_t)s * (CP + 4) + CP + 1] * __expf(pr[(size_t)s * (CP + 4) + CP] - mm);
  const float inv = l > 0.f ? 1.f / l : 0.f;
  for (int c = threadIdx.x * 2; c < CP; c += 512) {
    f32x2_t v = {0.f, 0.f};
#pragma unroll 4
    for (int s = 0; s < a.nsplit; ++s) {
      const float* p = pr + (size_t)s * (CP + 4);
      const float w = __expf(p[CP] - mm);
      const f32x2_t x = *reinterpret_cast<const f32x2_t*>(p + c);
      v.x = fmaf(x.x, w, v.x);
      v.y = fmaf(x.y, w, v.y);
    }
    *reinterpret_cast<uint32_t*>(reinterpret_cast<uint16_t*>(a.out) + row * CP + c) = pack_bf2(v.x * inv, v.y * inv);
  }
}

// f32: one workgroup per (head, row); 256 positions at a time, a thread scores one of them and then owns columns of
// the output.
__global__ __launch_bounds__(256) void latent_attn_f32_kernel(LatentAttnArgs a) {
  __shared__ __align__(16) float qs[TMX_MAX_LATENT_RANK + TMX_MAX_LATENT_ROT];
  __shared__ float ps[256], red[4];
  const int hd = blockIdx.x, m = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int seq = m / a.tpp, ld = a.rank_p + a.rot_p;
  const int step0 = max(min(*a.step, min(a.C, a.buf_len) - a.tpp), 0);
  const int limit = step0 + m % a.tpp;
  const size_t qrow = (size_t)m * a.H + hd;
  for (int i = tid; i < ld; i += 256) qs[i] = reinterpret_cast<const float*>(a.q)[qrow * ld + i];
  const float* cache = reinterpret_cast<const float*>(a.cache) + (size_t)seq * a.C * ld;
  const uint8_t* mrow = a.input_mask + (size_t)seq * a.buf_len;
  float mx = a.sink ? a.sink[hd] : -1e30f, l = a.sink ? 1.f : 0.f;
  float o[2] = {0.f, 0.f};
  __syncthreads();
  for (int p0 = 0; p0 <= limit; p0 += 256) {
    const int p = p0 + tid;
    const bool ok = p <= limit && mrow[p];
    float s = -1e30f;
    if (ok) {
      const float4* row = reinterpret_cast<const float4*>(cache + (size_t)p * ld);
      float d = 0.f;
      for (int i = 0; i < ld / 4; ++i) {
        const float4 k = row[i], qv = *reinterpret_cast<const float4*>(qs + 4 * i);
        d = fmaf(k.x, qv.x, d); d = fmaf(k.y, qv.y, d); d = fmaf(k.z, qv.z, d); d = fmaf(k.w, qv.w, d);
      }
      s = d * a.scale;
    }
    float top = wave_max(s);
    __syncthreads();  // the last chunk's ps and red are free
    if (lane == 0) red[wave] = top;
    __syncthreads();
    const float mn = fmaxf(mx, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
    const float alpha = expf(mx - mn);
    mx = mn;
    const float pr = ok ? expf(s - mn) : 0.f;
    ps[tid] = pr;
    const float sum = block_sum<4>(pr, red);  // its barriers also publish ps
    l = l * alpha + sum;
    const int n = min(256, limit - p0 + 1);
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int c = tid + 256 * i;
      if (c >= a.rank_p) continue;
      float v = o[i] * alpha;
      for (int j = 0; j < n; ++j) v = fmaf(ps[j], cache[(size_t)(p0 + j) * ld + c], v);
      o[i] = v;
    }
  }
  const float inv = l > 0.f ? 1.f / l : 0.f;
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int c = tid + 256 * i;
    if (c < a.rank_p) reinterpret_cast<float*>(a.out)[qrow * a.rank_p + c] = o[i] * inv;
  }
}

// ---------------------------------------------------------------------------
int latent_rows(hipStream_t st, int act, const LatentRowsArgs& a, int M) {
  if (M <= 0 || a.H <= 0 || a.rot <= 0 || a.rot % 2 || a.rot > a.rot_p || a.rank > a.rank_p || a.rank <= 0 ||
      !latent_attn_ok(a.rank_p, a.rot_p))
    return TMX_ERR_SHAPE;
  if (act == TMX_ACT_BF16) hipLaunchKernelGGL(latent_rows_kernel<uint16_t>, dim3(M), dim3(256), 0, st, a);
  else if (act == TMX_ACT_F32) hipLaunchKernelGGL(latent_rows_kernel<float>, dim3(M), dim3(256), 0, st, a);
  else return TMX_ERR_ARG;
  return check_launch();
}

bool latent_attn_ok(int rank_p, int rot_p) {
  return (rank_p == 64 || rank_p == 128 || rank_p == 256 || rank_p == 512) && (rot_p == 64 || rot_p == 128);
}

// A workgroup holds 64 or 128 query rows of a sequence, or 32 with its position groups on different blocks; the positions are split
// until every CU has a workgroup (one fits a CU at the full latent width).
struct LatentPlan { bool shared; int nsplit; };
constexpr int kLatentWgs = 256, kLatentMaxSplits = 32;
static int latent_block_rows(int rank_p, bool shared) { return !shared ? 32 : (rank_p > 256 ? 64 : 128); }
static LatentPlan latent_plan(int n_seq, int T, int H, int rank_p, int C) {
  LatentPlan p;
  const int rows = T * H;
  p.shared = rows > 32;
  const int per = latent_block_rows(rank_p, p.shared);
  const long wgs = (long)n_seq * ((rows + per - 1) / per);
  long ns = kLatentWgs / wgs;
  const int by_len = (C + 127) / 128;  // at least four blocks of 32 positions per split
  if (ns > by_len) ns = by_len;
  if (ns > kLatentMaxSplits) ns = kLatentMaxSplits;
  p.nsplit = ns < 1 ? 1 : (int)ns;
  return p;
}

size_t latent_attn_partial_bytes(int rows, int H, int rank_p) {
  // nsplit > 1 only while nsplit * workgroups <= kLatentWgs, and a workgroup holds at most 128 query rows
  size_t parts = (size_t)rows * H * kLatentMaxSplits;
  if (parts > (size_t)kLatentWgs * 128) parts = (size_t)kLatentWgs * 128;
  return parts * (rank_p + 4) * 4;
}

template <int KVT, int RT, bool SHARED>
static int launch_latent(hipStream_t st, const LatentAttnArgs& a) {
  using L = LatentShape<KVT, RT, SHARED>;
  static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(&latent_attn_kernel<KVT, RT, SHARED>),
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, (int)L::kBytes);
  if (attr != hipSuccess) return TMX_ERR_LAUNCH;
  const int per = 32 * L::WQ;
  hipLaunchKernelGGL((latent_attn_kernel<KVT, RT, SHARED>), dim3((a.tpp * a.H + per - 1) / per, a.n_seq, a.nsplit),
                     dim3(256), L::kBytes, st, a);
  return check_launch();
}
template <int KVT>
static int launch_latent_k(hipStream_t st, const LatentAttnArgs& a, bool shared) {
  if (a.rot_p == 64) return shared ? launch_latent<KVT, 1, true>(st, a) : launch_latent<KVT, 1, false>(st, a);
  return shared ? launch_latent<KVT, 2, true>(st, a) : launch_latent<KVT, 2, false>(st, a);
}

int latent_attention(hipStream_t st, int act, LatentAttnArgs a) {
  if (a.n_seq <= 0 || a.n_seq > 65535 || a.tpp <= 0 || a.H <= 0 || a.C <= 0 || a.tpp > a.C ||
      !latent_attn_ok(a.rank_p, a.rot_p))
    return TMX_ERR_SHAPE;
  if (act == TMX_ACT_F32) {
    if ((long)a.n_seq * a.tpp > 65535) return TMX_ERR_SHAPE;
    hipLaunchKernelGGL(latent_attn_f32_kernel, dim3(a.H, a.n_seq * a.tpp), dim3(256), 0, st, a);
    return check_launch();
  }
  if (act != TMX_ACT_BF16) return TMX_ERR_ARG;
  if ((size_t)a.C * (a.rank_p + a.rot_p) * 2 >= (1u << 31)) return TMX_ERR_SHAPE;
  const LatentPlan p = latent_plan(a.n_seq, a.tpp, a.H, a.rank_p, a.C);
  a.nsplit = p.nsplit;
  if (a.nsplit > 1 && !a.partial) return TMX_ERR_ARG;
  int rc;
  switch (a.rank_p) {
    case 64: rc = launch_latent_k<2>(st, a, p.shared); break;
    case 128: rc = launch_latent_k<4>(st, a, p.shared); break;
    case 256: rc = launch_latent_k<8>(st, a, p.shared); break;
    default: rc = launch_latent_k<16>(st, a, p.shared); break;
  }
  if (rc != TMX_OK || a.nsplit == 1) return rc;
  hipLaunchKernelGGL(latent_combine_kernel, dim3(a.n_seq * a.tpp * a.H), dim3(a.rank_p >= 512 ? 256 : (a.rank_p >= 256 ? 128 : 64)),
                     0, st, a);
  return check_launch();
}

}  // namespace tmx

using namespace tmx;

extern "C" int tmx_latent_rows(void* stream, int act, const void* z, int ldz, int off_qr, int off_kv,
                               const float* norm_w, float eps, const float* table, int positions_max,
                               const int32_t* positions, const int32_t* step, int buf_len, void* q, void* cache, int M,
                               int T, int H, int rot, int rank, int rank_p, int rot_p, int C) {
  if (!z || !table || !positions || !step || !q || (off_kv >= 0 && (!norm_w || !cache))) return TMX_ERR_ARG;
  LatentRowsArgs a = {};
  a.z = z; a.ldz = ldz; a.off_qr = off_qr; a.off_kv = off_kv; a.norm_w = norm_w; a.eps = eps; a.table = table;
  a.max_positions = positions_max; a.positions = positions; a.step = step; a.buf_len = buf_len; a.tpp = T;
  a.q = q; a.cache = cache; a.H = H; a.rot = rot; a.rank = rank; a.rank_p = rank_p; a.rot_p = rot_p; a.C = C;
  return latent_rows((hipStream_t)stream, act, a, M);
}

extern "C" size_t tmx_latent_attention_workspace_bytes(int n_seq, int T, int H, int rank_p, int C) {
  if (n_seq <= 0 || T <= 0 || H <= 0 || C <= 0) return 0;
  const LatentPlan p = latent_plan(n_seq, T, H, rank_p, C);
  return p.nsplit == 1 ? 0 : (size_t)n_seq * T * H * p.nsplit * (rank_p + 4) * 4;
}

extern "C" int tmx_latent_attention(void* stream, int act, const void* q, const void* cache, const float* sink,
                                    const uint8_t* input_mask, const int32_t* step, int buf_len, void* out,
                                    void* workspace, int n_seq, int T, int H, int rank_p, int rot_p, int C,
                                    float scale) {
  if (!q || !cache || !input_mask || !step || !out) return TMX_ERR_ARG;
  LatentAttnArgs a = {};
  a.q = q; a.cache = cache; a.sink = sink; a.input_mask = input_mask; a.step = step; a.buf_len = buf_len;
  a.out = out; a.partial = (float*)workspace; a.n_seq = n_seq; a.tpp = T; a.H = H; a.rank_p = rank_p;
  a.rot_p = rot_p; a.C = C; a.scale = scale;
  return latent_attention((hipStream_t)stream, act, a);
}
