// Grouped-query attention of dense models: query / key heads and value heads of their own widths, any number of query
// heads per key head, optionally a norm per head, a rotation of the first dimensions, chunks (a token sees the earlier
// tokens of its own chunk of positions) and a softmax sink.
//   head_rows_kernel      norm and rotation of queries and keys, cache rows, first visible slot of every row
//   head_attn_kernel      the walk over the cache on the matrix pipe (one or many tokens per sequence)
//   head_combine_kernel   merge of the splits of a query row
//   head_attn_f32_kernel  the same attention in f32 on the vector ALU
// The cache holds K [sequence][Kh][C][dk] and V [sequence][Kh][C][dv]: the rows one workgroup walks are consecutive.
#include "tmx_kernels.h"

namespace tmx {

__device__ __forceinline__ float act_get(const uint16_t* p) { return bf2f(*p); }
__device__ __forceinline__ float act_get(const float* p) { return *p; }
__device__ __forceinline__ void act_set(uint16_t* p, float v) { *p = f2bf(v); }
__device__ __forceinline__ void act_set(float* p, float v) { *p = v; }

// First slot of the chunk of the token at slot `col`.  Without unused slots in between it lies position - chunk start
// slots back; that guess is right when the slot holds a token at the chunk's first position, else the (never
// decreasing) positions are searched.
__device__ __forceinline__ int first_slot(const int32_t* pos, const uint8_t* mask, int col, int chunk) {
  if (chunk <= 0) return 0;
  const int p = max(pos[col], 0), start = p - p % chunk, guess = col - (p - start);
  if (guess >= 0 && mask[guess] && pos[guess] == start) return guess;
  int lo = 0, hi = col;  // the first slot in [lo, hi] whose position is at least `start`
  while (lo < hi) {
    const int mid = (lo + hi) >> 1;
    if (pos[mid] >= start) hi = mid;
    else lo = mid + 1;
  }
  return lo;
}

// A wave per head of a row: blockIdx.x = row * groups of 4 heads + group.
template <typename T>
__global__ __launch_bounds__(256) void head_rows_kernel(HeadRowsArgs a) {
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int heads = a.H + 2 * a.Kh, groups = (heads + 3) / 4;
  const int m = blockIdx.x / groups, hd = (blockIdx.x % groups) * 4 + wave;
  if (hd >= heads) return;
  const int tpp = a.tpp > 0 ? a.tpp : 1;
  const int seq = m / tpp, slot = min(*a.step + m % tpp, min(a.buf_len, a.C) - 1);
  const int32_t* prow = a.positions + (size_t)seq * a.buf_len;
  const T* z = reinterpret_cast<const T*>(a.z) + (size_t)m * a.ldz;
  if (hd >= a.H + a.Kh) {  // value head: copied
    const int g = hd - a.H - a.Kh;
    const T* src = z + (size_t)(a.H + a.Kh) * a.dk + (size_t)g * a.dv;
    T* dst = reinterpret_cast<T*>(a.vcache) + (((size_t)seq * a.Kh + g) * a.C + slot) * a.dv;
    for (int c = lane; c < a.dv; c += 64) dst[c] = src[c];
    return;
  }
  if (hd == 0 && lane == 0 && a.first) a.first[m] = first_slot(prow, a.input_mask + (size_t)seq * a.buf_len, slot, a.chunk);
  const int half = a.rot >> 1;
  const int pos = min(max(prow[slot], 0), a.max_positions - 1);
  const float2* tab = reinterpret_cast<const float2*>(a.table) + (size_t)pos * half;
  const bool key = hd >= a.H;
  const float* nw = key ? a.k_norm_w : a.q_norm_w;
  const T* src = z + (size_t)hd * a.dk;
  T* dst = key ? reinterpret_cast<T*>(a.kcache) + (((size_t)seq * a.Kh + hd - a.H) * a.C + slot) * a.dk
               : reinterpret_cast<T*>(a.q) + ((size_t)m * a.H + hd) * a.dk;
  constexpr int E = TMX_MAX_HEAD_DIM / 64;
  float v[E], u[E];  // this lane's values and their partners in the rotation
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < E; ++j) {
    const int c = lane + 64 * j;
    v[j] = u[j] = 0.f;
    if (c < a.dk) {
      v[j] = act_get(src + c);
      if (c < a.rot) u[j] = act_get(src + (c < half ? c + half : c - half));
    }
    ss += v[j] * v[j];
  }
  const float inv = nw ? 1.f / sqrtf(wave_sum(ss) / (float)a.dim + a.eps) : 1.f;
#pragma unroll
  for (int j = 0; j < E; ++j) {
    const int c = lane + 64 * j;
    if (c >= a.dk) continue;
    float o = v[j] * inv * (nw ? nw[c] : 1.f);
    if (c < a.rot) {
      const int i = c < half ? c : c - half, p = c < half ? c + half : i;
      const float w = u[j] * inv * (nw ? nw[p] : 1.f);
      const float2 cs = tab[i];
      o = c < half ? o * cs.x - w * cs.y : o * cs.x + w * cs.y;
    }
    act_set(dst + c, o);
  }
}

// ---------------------------------------------------------------------------
// The walk.  Query rows of a (sequence, kv head) are its (token, query head of the group) pairs, 32 of them the columns
// of an MFMA tile: scores^T [position, query] = K . Q^T and out^T [column, query] += V^T . P^T, a lane owning one query.
// 32 rows of K and of V go global -> LDS by direct loads (16-byte chunks XOR-swizzled by row); K is read by rows, V
// through the transposing LDS read.  Probabilities enter the product as bf16 hi + lo.
//   SHARED (many query rows): the four waves hold different query rows and walk the same blocks, double-buffered;
//   else (up to 32 query rows): the waves hold the same rows and walk different blocks in tiles of their own, and meet
//   through LDS at the end.
// KT, VT: padded widths / 64.
template <int KT, int VT, bool SHARED>
struct HeadShape {
  static constexpr int DK = KT * 64, DV = VT * 64;
  static constexpr int WQ = SHARED ? 4 : 1, WP = SHARED ? 1 : 4;
  static constexpr int kTile = 32 * (DK + DV);  // elements: K rows, then V rows
  static constexpr int kBufs = SHARED || kTile * 2 * 4 * 2 <= 64 * 1024 ? 2 : 1;
  static constexpr size_t kTiles = (size_t)kBufs * WP * kTile * 2;
  static constexpr size_t kMerge = SHARED ? 0 : (size_t)2 * (DV * 32 * 4 + 2 * 32 * 4);
  static constexpr size_t kBytes = kTiles > kMerge ? kTiles : kMerge;
};

// 16-byte chunk c of row r lies at chunk c ^ swz(r); CPR: chunks per row.  Rows of at least 256 bytes are told apart by
// four bits of the row, rows of 128 bytes (which alternate between the halves of the banks by themselves) by three.
template <int CPR>
__device__ __forceinline__ constexpr int head_swz(int row) {
  return CPR % 16 == 0 ? ((row & 3) << 2) | ((row >> 2) & 3) : (((row >> 1) & 1) << 2) | ((row >> 2) & 3);
}

template <int KT, int VT, bool SHARED>
__global__ __launch_bounds__(256, (KT + VT > 4 ? 1 : 2)) void head_attn_kernel(HeadAttnArgs a) {
  using SH = HeadShape<KT, VT, SHARED>;
  extern __shared__ __align__(16) unsigned char ha_smem[];
  constexpr int DK = SH::DK, DV = SH::DV, CK = DK / 8, CV = DV / 8, KS = DK / 16, VC = DV / 32;
  constexpr int WPW = 4 / SH::WP;  // waves that share a tile
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int h = lane >> 5, qi = lane & 31;
  const int wq = SHARED ? wave : 0, wp = SHARED ? 0 : wave, wg = SHARED ? wave : 0;
  const int G = a.H / a.Kh, rows = a.tpp * G;  // query rows of a (sequence, kv head)
  const int qblocks = (rows + 32 * SH::WQ - 1) / (32 * SH::WQ);
  const int pair = blockIdx.x / qblocks, q0 = (blockIdx.x % qblocks) * (32 * SH::WQ), split = blockIdx.z;
  const int seq = pair / a.Kh, kvh = pair % a.Kh;
  const int qr = q0 + wq * 32 + qi, qr_l = qr < rows ? qr : rows - 1;
  const int tok = qr_l / G, head = kvh * G + qr_l % G;
  const size_t qrow = ((size_t)seq * a.tpp + tok) * a.H + head;

  const __amdgpu_buffer_rsrc_t rk = make_rsrc(reinterpret_cast<const uint16_t*>(a.kcache) + (size_t)pair * a.C * DK, (uint32_t)a.C * DK * 2u);
  const __amdgpu_buffer_rsrc_t rv = make_rsrc(reinterpret_cast<const uint16_t*>(a.vcache) + (size_t)pair * a.C * DV, (uint32_t)a.C * DV * 2u);
  uint16_t* tiles = reinterpret_cast<uint16_t*>(ha_smem) + wp * SH::kBufs * SH::kTile;
  // 1 KiB per load, shared by WPW waves: load ld covers 64 chunks, this lane's lies at byte `off` of the 32 rows
  constexpr int kLk = DK / 16 / WPW, kLv = DV / 16 / WPW;
  int koff[kLk], voff[kLv];
#pragma unroll
  for (int i = 0; i < kLk; ++i) {
    const int g = (wg + WPW * i) * 64 + lane, row = g / CK, slot = g % CK;
    koff[i] = (row * CK + (slot ^ head_swz<CK>(row))) * 16;
  }
#pragma unroll
  for (int i = 0; i < kLv; ++i) {
    const int g = (wg + WPW * i) * 64 + lane, row = g / CV, slot = g % CV;
    voff[i] = (row * CV + (slot ^ head_swz<CV>(row))) * 16;
  }
  auto fetch = [&](int blk, int buf) __attribute__((always_inline)) {
    uint16_t* kt = tiles + buf * SH::kTile;
#pragma unroll
    for (int i = 0; i < kLk; ++i) load_row_to_lds(rk, kt + (wg + WPW * i) * 512, koff[i], blk * (32 * DK * 2));
#pragma unroll
    for (int i = 0; i < kLv; ++i) load_row_to_lds(rv, kt + 32 * DK + (wg + WPW * i) * 512, voff[i], blk * (32 * DV * 2));
  };
  const uint8_t* mrow = a.input_mask + (size_t)seq * a.buf_len;
  auto mask_byte = [&](int blk) __attribute__((always_inline)) {
    const int p = blk * 32 + qi;
    return (h == 0 && p < a.buf_len) ? mrow[p] : (uint8_t)0;
  };

  const int step0 = max(min(*a.step, min(a.C, a.buf_len) - a.tpp), 0);  // clamped: every slot read lies in the cache
  const int32_t* frow = a.first + (size_t)seq * a.tpp;
  const int first = max(frow[tok], 0);                        // oldest slot this query sees (it does not decrease along the tokens)
  const int b_beg = max(frow[q0 / G], 0) >> 5;                // blocks of the workgroup
  u32x4_t qf[KS];
  {
    const uint16_t* qp = reinterpret_cast<const uint16_t*>(a.q) + qrow * DK + (DK / 2) * h;
#pragma unroll
    for (int t = 0; t < KS; ++t) qf[t] = *reinterpret_cast<const u32x4_t*>(qp + 8 * t);
  }
  const int limit = step0 + tok;                              // newest slot this query sees
  const int limit0 = step0 + min(q0 + wq * 32, rows - 1) / G;  // the smallest one in the wave
  const int first1 = __shfl(first, 31, 64);                   // the largest one in the wave
  const int b_end = (step0 + (min(q0 + 32 * SH::WQ, rows) - 1) / G + 32) >> 5;

  f32x16_t o[VC];
#pragma unroll
  for (int c = 0; c < VC; ++c)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[c][r] = 0.f;
  // running maximum and sum of the softmax; exponentials are powers of two throughout (scores times log2 e), a masked
  // score is far below the maximum of a row that has seen none
  constexpr float kLog2e = 1.44269504f, kUnseen = -1e30f, kHidden = -2e30f;
  const float scale2 = a.scale * kLog2e;
  float m = kUnseen, l = 0.f;

  // scaled scores of a block; the largest one of this lane's query in mn
  auto scores = [&](const uint16_t* kt, int blk, uint32_t mbits, f32x16_t& sacc, float& mn) __attribute__((always_inline)) {
    const int sw = head_swz<CK>(qi);
#pragma unroll
    for (int r = 0; r < 16; ++r) sacc[r] = 0.f;
#pragma unroll
    for (int t = 0; t < KS; ++t) {  // lane (position, h) multiplies the half h of its row
      const bf16x8_t kf = *reinterpret_cast<const bf16x8_t*>(kt + qi * DK + (((KS * h + t) ^ sw) << 3));
      sacc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, __builtin_bit_cast(bf16x8_t, qf[t]), sacc, 0, 0, 0);
    }
    mn = kUnseen;
    if (mbits == 0xFFFFFFFFu && blk * 32 + 31 <= limit0 && blk * 32 >= first1) {  // every query of the wave sees the whole block
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        sacc[r] *= scale2;
        mn = fmaxf(mn, sacc[r]);
      }
    } else {
      const int lim = limit - blk * 32 - 4 * h, low = first - blk * 32 - 4 * h;
      const uint32_t mb2 = mbits >> (4 * h);
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int pc = (r >> 2) * 8 + (r & 3);  // acc_row(r, lane) without the lane's half
        sacc[r] = pc <= lim && pc >= low && ((mb2 >> pc) & 1u) ? sacc[r] * scale2 : kHidden;
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
      for (int c = 0; c < VC; ++c)
#pragma unroll
        for (int r = 0; r < 16; ++r) o[c][r] *= alpha;
    }
  };
  // transposed fragments of the output product: lane (column 32 c + qi, h) takes two runs of four consecutive rows (see
  // gqa_tile_walk); in assembly, because for the builtin the compiler waits for every direct-to-LDS load in flight
  const int k4 = (lane & 15) >> 2, q4 = lane & 3, g2 = (lane >> 4) & 1;
  const uint32_t lsw = ((2 * g2 + (q4 >> 1)) ^ head_swz<CV>(4 * h + k4)) * 16;
  const uint32_t vbase = (32 * DK + (4 * h + k4) * DV + 4 * (q4 & 1)) * 2;
  constexpr int R = 4;  // fragments in flight
  u32x2_t vf[R][2];
  auto load_v = [&](uint32_t vb, auto fc) __attribute__((always_inline)) {
    constexpr int f = decltype(fc)::value, kb2 = f / VC, c = f % VC;
    static_for<2>([&](auto ac) __attribute__((always_inline)) {
      constexpr int row0 = 16 * kb2 + 8 * decltype(ac)::value;
      const uint32_t ad = vb + (lsw ^ (uint32_t)(((4 * c) ^ head_swz<CV>(row0)) * 16));
      u32x2_t& dst = vf[f % R][decltype(ac)::value];
      asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(dst) : "v"(ad), "i"(row0 * DV * 2));
    });
  };
  auto lds_addr = [](const uint16_t* p) __attribute__((always_inline)) {
    return (uint32_t)(uintptr_t)(__attribute__((address_space(3))) const uint16_t*)p;
  };
  auto block = [&](int blk, uint32_t mbits, int buf) __attribute__((always_inline)) {
    const uint16_t* kt = tiles + buf * SH::kTile;
    const uint32_t vb = lds_addr(kt) + vbase;
    f32x16_t sacc;
    float mn;
    u32x4_t p[4];  // probabilities as bf16 hi (p[0], p[1]) and lo (p[2], p[3]), 16 positions each
    scores(kt, blk, mbits, sacc, mn);
    static_for<R>([&](auto fc) __attribute__((always_inline)) { load_v(vb, fc); });  // they do not wait for the softmax
    __builtin_amdgcn_sched_barrier(0);
    move_reference(mn);
#pragma unroll
    for (int r = 0; r < 16; r += 2) {
      const float p0 = __builtin_amdgcn_exp2f(sacc[r] - m), p1 = __builtin_amdgcn_exp2f(sacc[r + 1] - m);
      const uint32_t hi = pack_bf2(p0, p1);
      p[r >> 3][(r >> 1) & 3] = hi;
      p[2 + (r >> 3)][(r >> 1) & 3] = pack_bf2(p0 - bf_lo(hi), p1 - bf_hi(hi));
      l += p0 + p1;
    }
    // out^T += V^T . P^T, 16 positions (accumulator registers 8 kb2 .. 8 kb2 + 7) per MFMA
    static_for<2 * VC>([&](auto fc) __attribute__((always_inline)) {
      constexpr int f = decltype(fc)::value, kb2 = f / VC, c = f % VC;
      constexpr int kLater = 2 * VC - 1 - f < R - 1 ? 2 * VC - 1 - f : R - 1;  // fragments requested behind this one
      u32x2_t &v0 = vf[f % R][0], &v1 = vf[f % R][1];
      asm volatile("s_waitcnt lgkmcnt(%2)" : "+v"(v0), "+v"(v1) : "i"(2 * kLater));
      const u32x4_t v = {v0.x, v0.y, v1.x, v1.y};
      o[c] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, v), __builtin_bit_cast(bf16x8_t, p[kb2]),
                                                     o[c], 0, 0, 0);
      o[c] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, v),
                                                     __builtin_bit_cast(bf16x8_t, p[2 + kb2]), o[c], 0, 0, 0);
      if constexpr (f + R < 2 * VC) load_v(vb, IC<f + R>{});
      __builtin_amdgcn_sched_barrier(0);
    });
  };

  if constexpr (SHARED) {
    const int blk0 = b_beg + split;
    const int rounds = b_end > blk0 ? (b_end - blk0 + a.nsplit - 1) / a.nsplit : 0;  // the same in every wave
    uint8_t mb = mask_byte(blk0);
    if (rounds > 0) fetch(blk0, 0);
    for (int round = 0; round < rounds; ++round) {
      const int blk = blk0 + round * a.nsplit, buf = round & 1;
      const uint32_t mbits = (uint32_t)__ballot(mb != 0);
      __builtin_amdgcn_s_waitcnt(0x0F70);  // this round's tile has landed
      __syncthreads();                     // ... in every wave, and the other buffer's readers are done
      mb = mask_byte(blk + a.nsplit);
      if (round + 1 < rounds) fetch(blk + a.nsplit, buf ^ 1);
      block(blk, mbits, buf);
    }
  } else {
    const int stride = a.nsplit * SH::WP;
    int blk = b_beg + split * SH::WP + wp, buf = 0;
    uint8_t mb = mask_byte(blk);
    if (blk < b_end) fetch(blk, 0);
    for (; blk < b_end; blk += stride) {
      const uint32_t mbits = (uint32_t)__ballot(mb != 0);
      __builtin_amdgcn_s_waitcnt(0x0F70);  // the wave's own tile has landed
      __builtin_amdgcn_sched_barrier(0);
      mb = mask_byte(blk + stride);
      const bool more = blk + stride < b_end;
      if (SH::kBufs == 2 && more) fetch(blk + stride, buf ^ 1);
      block(blk, mbits, buf);
      if (SH::kBufs == 2) buf ^= 1;
      else if (more) {
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // the tile's reads are complete
        fetch(blk + stride, 0);
      }
    }
  }
  l += __shfl_xor(l, 32, 64);
  if constexpr (!SHARED) {
    // merge the waves: the upper half of them hands its state to the lower half, until one is left
    constexpr int kPart = DV * 32;
    float* mf = reinterpret_cast<float*>(ha_smem);
    float* ml = mf + 2 * kPart;  // [slot][m, l][32]
    auto put = [&](int s) __attribute__((always_inline)) {
#pragma unroll
      for (int c = 0; c < VC; ++c)
#pragma unroll
        for (int r = 0; r < 16; ++r) mf[s * kPart + ((c * 16 + r) << 6) + lane] = o[c][r];
      if (h == 0) {
        ml[s * 64 + qi] = m;
        ml[s * 64 + 32 + qi] = l;
      }
    };
    auto take = [&](int s) __attribute__((always_inline)) {
      const float m2 = ml[s * 64 + qi], l2 = ml[s * 64 + 32 + qi];
      const float mm = fmaxf(m, m2), w1 = __builtin_amdgcn_exp2f(m - mm), w2 = __builtin_amdgcn_exp2f(m2 - mm);
#pragma unroll
      for (int c = 0; c < VC; ++c)
#pragma unroll
        for (int r = 0; r < 16; ++r) o[c][r] = o[c][r] * w1 + mf[s * kPart + ((c * 16 + r) << 6) + lane] * w2;
      l = l * w1 + l2 * w2;
      m = mm;
    };
#pragma unroll
    for (int n = 2; n > 0; n >>= 1) {
      __syncthreads();
      if (wp >= n && wp < 2 * n) put(wp - n);
      __syncthreads();
      if (wp < n) take(wp);
    }
    if (wp != 0) return;
  }
  if (qr >= rows) return;
  if (a.nsplit == 1) {
    float w = 1.f;
    if (a.sink) {  // one more term of the denominator, without a value
      const float s = a.sink[head] * kLog2e, mm = fmaxf(m, s);
      w = __builtin_amdgcn_exp2f(m - mm);
      l = l * w + __builtin_amdgcn_exp2f(s - mm);
    }
    const float inv = l > 0.f ? w / l : 0.f;
    uint16_t* out = reinterpret_cast<uint16_t*>(a.out);
    const int row = seq * a.tpp + tok;
#pragma unroll
    for (int c = 0; c < VC; ++c)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        uint2 v;
        v.x = pack_bf2(o[c][4 * i] * inv, o[c][4 * i + 1] * inv);
        v.y = pack_bf2(o[c][4 * i + 2] * inv, o[c][4 * i + 3] * inv);
        const int col = head * DV + 32 * c + 8 * i + 4 * h;
        *reinterpret_cast<uint2*>(out + (a.out_tiled ? act_tile_off(row, col, a.H * DV) : (size_t)row * a.H * DV + col)) = v;
      }
    return;
  }
  float* pr = a.partial + (qrow * a.nsplit + split) * (DV + 4);
#pragma unroll
  for (int c = 0; c < VC; ++c)
#pragma unroll
    for (int i = 0; i < 4; ++i)
      *reinterpret_cast<f32x4_t*>(pr + 32 * c + 8 * i + 4 * h) = f32x4_t{o[c][4 * i], o[c][4 * i + 1], o[c][4 * i + 2], o[c][4 * i + 3]};
  if (h == 0) {
    pr[DV] = m * (1.f / kLog2e);  // (natural units, as the sink)
    pr[DV + 1] = l;
  }
}

// A wave per (row, head): the softmax-weighted sum of its splits, then the sink.
__global__ __launch_bounds__(256) void head_combine_kernel(HeadAttnArgs a, int total) {
  const int qrow = blockIdx.x * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (qrow >= total) return;
  const int DV = a.dv, ns = a.nsplit, row = qrow / a.H, head = qrow % a.H;
  const float* pr = a.partial + (size_t)qrow * ns * (DV + 4);  // [split][DV values | max | sum | -]
  // lane s holds the maximum and the sum of split s (at most 32 of them)
  float pm = lane < ns ? pr[(size_t)lane * (DV + 4) + DV] : -1e30f, pl = lane < ns ? pr[(size_t)lane * (DV + 4) + DV + 1] : 0.f;
  const float sink = a.sink ? a.sink[head] : -1e30f, mm = fmaxf(wave_max(pm), sink);
  const float w = __expf(pm - mm), l = wave_sum(pl * w) + (a.sink ? __expf(sink - mm) : 0.f);
  const float inv = l > 0.f ? 1.f / l : 0.f;
  for (int c = lane * 2; c < DV; c += 128) {
    f32x2_t v = {0.f, 0.f};
    for (int s0 = 0; s0 < ns; s0 += 4) {  // four parts requested at a time (clamped), added in ascending order
      f32x2_t x[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) x[u] = *reinterpret_cast<const f32x2_t*>(pr + (size_t)min(s0 + u, ns - 1) * (DV + 4) + c);
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const float ws = s0 + u < ns ? __shfl(w, s0 + u, 64) : 0.f;
        v.x = fmaf(x[u].x, ws, v.x);
        v.y = fmaf(x[u].y, ws, v.y);
      }
    }
    const int col = head * DV + c;
    *reinterpret_cast<uint32_t*>(reinterpret_cast<uint16_t*>(a.out) +
                                 (a.out_tiled ? act_tile_off(row, col, a.H * DV) : (size_t)row * a.H * DV + col)) = pack_bf2(v.x * inv, v.y * inv);
  }
}

// f32: one workgroup per (head, row); 256 positions at a time, a thread scores one of them and then owns one column of
// the output.
__global__ __launch_bounds__(256) void head_attn_f32_kernel(HeadAttnArgs a) {
  __shared__ __align__(16) float qs[TMX_MAX_HEAD_DIM];
  __shared__ float ps[256], red[4];
  const int hd = blockIdx.x, row = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int seq = row / a.tpp, kvh = hd / (a.H / a.Kh);
  const int step0 = max(min(*a.step, min(a.C, a.buf_len) - a.tpp), 0);
  const int limit = step0 + row % a.tpp, first = max(a.first[row], 0);
  const size_t qrow = (size_t)row * a.H + hd, pair = (size_t)seq * a.Kh + kvh;
  for (int i = tid; i < a.dk; i += 256) qs[i] = reinterpret_cast<const float*>(a.q)[qrow * a.dk + i];
  const float* kc = reinterpret_cast<const float*>(a.kcache) + pair * a.C * a.dk;
  const float* vc = reinterpret_cast<const float*>(a.vcache) + pair * a.C * a.dv;
  const uint8_t* mrow = a.input_mask + (size_t)seq * a.buf_len;
  float mx = a.sink ? a.sink[hd] : -1e30f, l = a.sink ? 1.f : 0.f, o = 0.f;
  __syncthreads();
  for (int p0 = first; p0 <= limit; p0 += 256) {
    const int p = p0 + tid;
    const bool ok = p <= limit && mrow[p];
    float s = -1e30f;
    if (ok) {
      const float4* kr = reinterpret_cast<const float4*>(kc + (size_t)p * a.dk);
      float d = 0.f;
      for (int i = 0; i < a.dk / 4; ++i) {
        const float4 k = kr[i], qv = *reinterpret_cast<const float4*>(qs + 4 * i);
        d = fmaf(k.x, qv.x, d); d = fmaf(k.y, qv.y, d); d = fmaf(k.z, qv.z, d); d = fmaf(k.w, qv.w, d);
      }
      s = d * a.scale;
    }
    const float top = wave_max(s);
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
    if (tid < a.dv) {
      float v = o * alpha;
      for (int j = 0; j < n; ++j) v = fmaf(ps[j], vc[(size_t)(p0 + j) * a.dv + tid], v);
      o = v;
    }
  }
  if (tid < a.dv) reinterpret_cast<float*>(a.out)[qrow * a.dv + tid] = l > 0.f ? o / l : 0.f;
}

// ---------------------------------------------------------------------------
bool head_attn_ok(int dk, int dv) {
  auto ok = [](int d) { return d == 64 || d == 128 || d == 256; };
  return ok(dk) && ok(dv);
}

int head_rows(hipStream_t st, int act, const HeadRowsArgs& a, int M) {
  if (M <= 0 || a.H <= 0 || a.Kh <= 0 || a.H % a.Kh || a.dim <= 0 || a.dim > a.dk || a.rot < 0 || a.rot % 2 || a.rot > a.dim ||
      a.C <= 0 || a.chunk < 0 || !head_attn_ok(a.dk, a.dv))
    return TMX_ERR_SHAPE;
  const long wgs = (long)M * ((a.H + 2 * a.Kh + 3) / 4);
  if (wgs > 0x7FFFFFFF) return TMX_ERR_SHAPE;
  if (act == TMX_ACT_BF16) hipLaunchKernelGGL(head_rows_kernel<uint16_t>, dim3(wgs), dim3(256), 0, st, a);
  else if (act == TMX_ACT_F32) hipLaunchKernelGGL(head_rows_kernel<float>, dim3(wgs), dim3(256), 0, st, a);
  else return TMX_ERR_ARG;
  return check_launch();
}

// A workgroup holds 128 query rows of a (sequence, kv head), or up to 32 with its waves on different blocks; the slots a
// row sees are split until the CUs are full, as long as a split keeps its waves busy for a while.
struct HeadPlan { bool shared; int nsplit; };
constexpr int kHeadWgs = 512, kHeadMaxSplits = 32, kHeadSplitSlots = 256;
static HeadPlan head_plan(int n_seq, int T, int H, int Kh, int C, int chunk) {
  HeadPlan p;
  const int rows = T * (H / Kh);
  p.shared = rows > 32;
  const int per = p.shared ? 128 : 32;
  const long wgs = (long)n_seq * Kh * ((rows + per - 1) / per);
  long ns = kHeadWgs / wgs;
  long seen = chunk > 0 && (long)chunk + T < C ? (long)chunk + T : C;  // slots a workgroup walks at most
  const int by_len = (int)((seen + kHeadSplitSlots - 1) / kHeadSplitSlots);
  if (ns > by_len) ns = by_len;
  if (ns > kHeadMaxSplits) ns = kHeadMaxSplits;
  p.nsplit = ns < 1 ? 1 : (int)ns;
  return p;
}

size_t head_attn_partial_bytes(int rows, int H, int dv) {
  // nsplit > 1 only while nsplit * workgroups <= kHeadWgs, and a workgroup holds at most 128 query rows
  size_t parts = (size_t)rows * H * kHeadMaxSplits;
  if (parts > (size_t)kHeadWgs * 128) parts = (size_t)kHeadWgs * 128;
  return parts * (dv + 4) * 4;
}

template <int KT, int VT, bool SHARED>
static int launch_head(hipStream_t st, const HeadAttnArgs& a) {
  using L = HeadShape<KT, VT, SHARED>;
  static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(&head_attn_kernel<KT, VT, SHARED>),
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, (int)L::kBytes);
  if (attr != hipSuccess) return TMX_ERR_LAUNCH;
  const int rows = a.tpp * (a.H / a.Kh), per = 32 * L::WQ;
  hipLaunchKernelGGL((head_attn_kernel<KT, VT, SHARED>), dim3((size_t)a.n_seq * a.Kh * ((rows + per - 1) / per), 1, a.nsplit),
                     dim3(256), L::kBytes, st, a);
  return check_launch();
}
template <int KT>
static int launch_head_v(hipStream_t st, const HeadAttnArgs& a, bool shared) {
  switch (a.dv) {
    case 64: return shared ? launch_head<KT, 1, true>(st, a) : launch_head<KT, 1, false>(st, a);
    case 128: return shared ? launch_head<KT, 2, true>(st, a) : launch_head<KT, 2, false>(st, a);
    default: return shared ? launch_head<KT, 4, true>(st, a) : launch_head<KT, 4, false>(st, a);
  }
}

int head_attention(hipStream_t st, int act, HeadAttnArgs a) {
  if (a.n_seq <= 0 || a.tpp <= 0 || a.H <= 0 || a.Kh <= 0 || a.H % a.Kh || a.C <= 0 || a.tpp > a.C || a.tpp > a.buf_len ||
      a.chunk < 0 || !head_attn_ok(a.dk, a.dv) || (long)a.n_seq * a.tpp * a.H > 0x3FFFFFFF)
    return TMX_ERR_SHAPE;
  if (act == TMX_ACT_F32) {
    if ((long)a.n_seq * a.tpp > 65535) return TMX_ERR_SHAPE;
    hipLaunchKernelGGL(head_attn_f32_kernel, dim3(a.H, a.n_seq * a.tpp), dim3(256), 0, st, a);
    return check_launch();
  }
  if (act != TMX_ACT_BF16) return TMX_ERR_ARG;
  // buffer descriptors hold byte offsets of 31 bits
  if ((size_t)(a.C + 32 * 4 * kHeadMaxSplits) * (a.dk > a.dv ? a.dk : a.dv) * 2 >= (1u << 31)) return TMX_ERR_SHAPE;
  if (a.out_tiled && a.n_seq * a.tpp > 128) return TMX_ERR_ARG;
  const HeadPlan p = head_plan(a.n_seq, a.tpp, a.H, a.Kh, a.C, a.chunk);
  a.nsplit = p.nsplit;
  if (a.nsplit > 1 && !a.partial) return TMX_ERR_ARG;
  int rc;
  switch (a.dk) {
    case 64: rc = launch_head_v<1>(st, a, p.shared); break;
    case 128: rc = launch_head_v<2>(st, a, p.shared); break;
    default: rc = launch_head_v<4>(st, a, p.shared); break;
  }
  if (rc != TMX_OK || a.nsplit == 1) return rc;
  const int total = a.n_seq * a.tpp * a.H;
  hipLaunchKernelGGL(head_combine_kernel, dim3((total + 3) / 4), dim3(256), 0, st, a, total);
  return check_launch();
}

}  // namespace tmx

using namespace tmx;

extern "C" int tmx_head_rows(void* stream, int act, const void* z, int ldz, const float* q_norm_w, const float* k_norm_w,
                             float eps, const float* table, int positions_max, const int32_t* positions,
                             const uint8_t* input_mask, const int32_t* step, int buf_len, void* q, void* kcache,
                             void* vcache, int32_t* first, int M, int T, int H, int Kh, int dim, int dk, int dv, int rot,
                             int C, int chunk) {
  if (!z || !positions || !input_mask || !step || !q || !kcache || !vcache || !first || (rot > 0 && !table)) return TMX_ERR_ARG;
  if (T <= 0 || M % T || positions_max <= 0 || buf_len <= 0) return TMX_ERR_SHAPE;
  HeadRowsArgs a = {};
  a.z = z; a.ldz = ldz; a.q_norm_w = q_norm_w; a.k_norm_w = k_norm_w; a.eps = eps;
  a.table = table; a.max_positions = positions_max; a.positions = positions; a.input_mask = input_mask; a.step = step;
  a.buf_len = buf_len; a.tpp = T; a.q = q; a.kcache = kcache; a.vcache = vcache; a.first = first;
  a.H = H; a.Kh = Kh; a.dim = dim; a.dk = dk; a.dv = dv; a.rot = rot; a.C = C; a.chunk = chunk;
  return head_rows((hipStream_t)stream, act, a, M);
}

extern "C" size_t tmx_head_attention_workspace_bytes(int n_seq, int T, int H, int Kh, int dv, int C, int chunk) {
  if (n_seq <= 0 || T <= 0 || H <= 0 || Kh <= 0 || H % Kh || C <= 0) return 0;
  const HeadPlan p = head_plan(n_seq, T, H, Kh, C, chunk);
  return p.nsplit == 1 ? 0 : (size_t)n_seq * T * H * p.nsplit * (dv + 4) * 4;
}

extern "C" int tmx_head_attention(void* stream, int act, const void* q, const void* kcache, const void* vcache,
                                  const float* sink, const int32_t* first, const uint8_t* input_mask, const int32_t* step,
                                  int buf_len, void* out, void* workspace, int n_seq, int T, int H, int Kh, int dk, int dv,
                                  int C, int chunk, float scale) {
  if (!q || !kcache || !vcache || !first || !input_mask || !step || !out) return TMX_ERR_ARG;
  HeadAttnArgs a = {};
  a.q = q; a.kcache = kcache; a.vcache = vcache; a.sink = sink; a.first = first; a.input_mask = input_mask; a.step = step;
  a.buf_len = buf_len; a.out = out; a.partial = (float*)workspace; a.n_seq = n_seq; a.tpp = T; a.H = H; a.Kh = Kh;
  a.dk = dk; a.dv = dv; a.C = C; a.chunk = chunk; a.scale = scale;
  return head_attention((hipStream_t)stream, act, a);
}
