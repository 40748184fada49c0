// Grouped-query attention of dense models: query / key heads and value heads of their own widths, any number of query
// heads per key head, optionally a norm per head, a rotation of the first dimensions, chunks (a token sees the earlier
// tokens of its own chunk of positions) and a softmax sink.
//   row_places_kernel     first slot every row sees and its position, once per pass and chunk size
//   head_rows_kernel      norm and rotation of queries and keys, cache rows
//   head_attn_kernel      the walk over the cache on the matrix pipe (one or many tokens per sequence); for one token per
//                         sequence the row part is in front of it in the same launch
//   head_combine_kernel   merge of the splits of a query row
//   head_attn_f32_kernel  the same attention in f32 on the vector ALU
// The cache holds K [sequence][Kh][C][dk] and V [sequence][Kh][C][dv]: the rows one workgroup walks are consecutive.
#include "tmx_kernels.h"

namespace tmx {

__device__ __forceinline__ float act_get(const uint16_t* p) { return bf2f(*p); }
__device__ __forceinline__ float act_get(const float* p) { return *p; }

// First slot of the chunk of the token at slot `col`.  Without unused slots in between it lies position - chunk start
// slots back; that guess is right when the slot holds a token at the chunk's first position, else the (never
// decreasing) positions are searched.
__device__ __forceinline__ int first_slot(const int32_t* pos, const uint8_t* mask, int col, int chunk) {
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

__global__ __launch_bounds__(256) void row_places_kernel(RowPlacesArgs a, int M) {
  const int m = blockIdx.x * 256 + threadIdx.x;
  if (m >= M) return;
  const int seq = m / a.tpp, slot = min(*a.step + m % a.tpp, min(a.buf_len, a.C) - 1);
  const size_t off = (size_t)seq * a.buf_len;
  const int first = a.chunk > 0 ? first_slot(a.positions + off, a.input_mask + off, slot, a.chunk) : 0;
  a.place[m] = make_int2(first, max(a.positions[off + slot], 0));
}

// E consecutive values of an act tensor at an offset that is a multiple of E.
template <int E>
__device__ __forceinline__ void load_e(const uint16_t* p, float* v) {
  if constexpr (E == 1) {
    v[0] = bf2f(*p);
  } else {
#pragma unroll
    for (int i = 0; i < E / 2; ++i) {
      const uint32_t w = reinterpret_cast<const uint32_t*>(p)[i];
      v[2 * i] = bf_lo(w);
      v[2 * i + 1] = bf_hi(w);
    }
  }
}
template <int E>
__device__ __forceinline__ void load_e(const float* p, float* v) {
#pragma unroll
  for (int i = 0; i < E; ++i) v[i] = p[i];
}
template <int E>
__device__ __forceinline__ void store_e(uint16_t* p, const float* v) {
  if constexpr (E == 1) {
    *p = f2bf(v[0]);
  } else {
#pragma unroll
    for (int i = 0; i < E / 2; ++i) reinterpret_cast<uint32_t*>(p)[i] = pack_bf2(v[2 * i], v[2 * i + 1]);
  }
}
template <int E>
__device__ __forceinline__ void store_e(float* p, const float* v) {
#pragma unroll
  for (int i = 0; i < E; ++i) p[i] = v[i];
}

// What a lane needs of the rotation at one position: it owns the E columns c = E lane .. of a head of 64 E columns, with
// partners p (a column past the rotated ones is its own).  The loads are free of branches, so that those of several heads
// are in flight together.
template <int E>
struct HeadLane {
  int c, p[E];
  float cs[E], sn[E];  // sn carries the sign of the column's half; 1, 0 past the rotated columns
  __device__ __forceinline__ HeadLane(const HeadRowsArgs& a, int lane, int pos) : c(E * lane) {
    const int rot = a.rot, half = rot >> 1;
    // (without a rotation the loads below read some 8 valid bytes)
    const float2* tab = rot > 0 ? reinterpret_cast<const float2*>(a.table) + (size_t)pos * half : reinterpret_cast<const float2*>(a.place);
    float2 t[E];
#pragma unroll
    for (int e = 0; e < E; ++e) {
      const int k = c + e;
      t[e] = tab[k < half ? k : (k < rot ? k - half : 0)];
      p[e] = k < half ? k + half : (k < rot ? k - half : k);
    }
#pragma unroll
    for (int e = 0; e < E; ++e) {
      const int k = c + e;
      cs[e] = k < rot ? t[e].x : 1.f;
      sn[e] = k < half ? -t[e].y : (k < rot ? t[e].y : 0.f);
    }
  }
  // a head's values of this lane: its own columns and their partners, with the norm's weights
  struct Head {
    float v[E], u[E], wv[E], wu[E];
  };
  template <typename T>
  __device__ __forceinline__ void load(Head& d, const T* src, const float* nw) const {
    load_e<E>(src + c, d.v);
    const float* w = nw ? nw : reinterpret_cast<const float*>(src);  // (without a norm the values read are not used)
#pragma unroll
    for (int e = 0; e < E; ++e) {
      d.u[e] = act_get(src + p[e]);
      d.wv[e] = w[c + e];
      d.wu[e] = w[p[e]];
    }
  }
  // the head's normed and rotated values
  __device__ __forceinline__ void finish(Head& d, bool norm, int dim, float eps) const {
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < E; ++e) ss += d.v[e] * d.v[e];
    const float inv = norm ? 1.f / sqrtf(wave_sum(ss) / (float)dim + eps) : 1.f;
#pragma unroll
    for (int e = 0; e < E; ++e)
      d.v[e] = d.v[e] * inv * (norm ? d.wv[e] : 1.f) * cs[e] + d.u[e] * inv * (norm ? d.wu[e] : 1.f) * sn[e];
  }
};

// Four heads of a row per wave: blockIdx.x = row * groups of 16 heads + group.  E: columns of a query / key head / 64.
template <typename T, int E>
__global__ __launch_bounds__(256) void head_rows_kernel(HeadRowsArgs a) {
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int heads = a.H + 2 * a.Kh, groups = (heads + 15) / 16, qk = a.H + a.Kh;
  const int m = blockIdx.x / groups, hd0 = (blockIdx.x % groups) * 16 + wave * 4;
  if (hd0 >= heads) return;
  const int tpp = a.tpp > 0 ? a.tpp : 1;
  const int seq = m / tpp, slot = min(*a.step + m % tpp, min(a.buf_len, a.C) - 1);
  const T* z = reinterpret_cast<const T*>(a.z) + (size_t)m * a.ldz;
  if (hd0 < qk) {
    const HeadLane<E> hl(a, lane, min(a.place[m].y, a.max_positions - 1));
    typename HeadLane<E>::Head d[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {  // (heads past the last key repeat it)
      const int hd = min(hd0 + i, qk - 1);
      hl.load(d[i], z + (size_t)hd * (64 * E), hd >= a.H ? a.k_norm_w : a.q_norm_w);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int hd = hd0 + i;
      if (hd >= qk) break;
      const bool key = hd >= a.H;
      hl.finish(d[i], key ? a.k_norm_w : a.q_norm_w, a.dim, a.eps);
      T* dst = key ? reinterpret_cast<T*>(a.kcache) + (((size_t)seq * a.Kh + hd - a.H) * a.C + slot) * (64 * E)
                   : reinterpret_cast<T*>(a.q) + ((size_t)m * a.H + hd) * (64 * E);
      store_e<E>(dst + hl.c, d[i].v);
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {  // value heads are copied
    const int g = hd0 + i - qk;
    if (g < 0 || g >= a.Kh) continue;
    const uint32_t* src = reinterpret_cast<const uint32_t*>(z + (size_t)qk * a.dk + (size_t)g * a.dv);
    uint32_t* dst = reinterpret_cast<uint32_t*>(reinterpret_cast<T*>(a.vcache) + (((size_t)seq * a.Kh + g) * a.C + slot) * a.dv);
    for (int c = lane; c < a.dv * (int)sizeof(T) / 4; c += 64) dst[c] = src[c];
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
//   ROWS (not SHARED, one token per sequence): the workgroup makes its queries and the new cache row from the fused
//   projection itself; they wait in LDS, from where the new row replaces what its slot held in the tile.
// KT, VT: padded widths / 64.
template <int KT, int VT, bool SHARED, bool ROWS>
struct HeadShape {
  static constexpr int DK = KT * 64, DV = VT * 64;
  static constexpr int WQ = SHARED ? 4 : 1, WP = SHARED ? 1 : 4;
  static constexpr int kTile = 32 * (DK + DV);  // elements: K rows, then V rows
  static constexpr int kBufs = SHARED || kTile * 2 * 4 * 2 <= 64 * 1024 ? 2 : 1;
  static constexpr size_t kTiles = (size_t)kBufs * WP * kTile * 2;
  static constexpr size_t kMerge = SHARED ? 0 : (size_t)2 * (DV * 32 * 4 + 2 * 32 * 4);
  static constexpr size_t kStage = (kTiles > kMerge ? kTiles : kMerge);  // queries [32][DK], key [DK], value [DV] bf16
  static constexpr size_t kBytes = kStage + (ROWS ? (size_t)(33 * DK + DV) * 2 : 0);
};

// 16-byte chunk c of row r lies at chunk c ^ swz(r); CPR: chunks per row.  Rows of at least 256 bytes are told apart by
// four bits of the row, rows of 128 bytes (which alternate between the halves of the banks by themselves) by three.
template <int CPR>
__device__ __forceinline__ constexpr int head_swz(int row) {
  return CPR % 16 == 0 ? ((row & 3) << 2) | ((row >> 2) & 3) : (((row >> 1) & 1) << 2) | ((row >> 2) & 3);
}

template <int KT, int VT, bool SHARED, bool ROWS>
__global__ __launch_bounds__(256, (KT + VT > 4 ? 1 : 2)) void head_attn_kernel(HeadAttnArgs a, HeadRowsArgs ra) {
  static_assert(!(SHARED && ROWS), "one token per sequence only");
  using SH = HeadShape<KT, VT, SHARED, ROWS>;
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
  auto fetch_k = [&](int blk, int buf) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < kLk; ++i) load_row_to_lds(rk, tiles + buf * SH::kTile + (wg + WPW * i) * 512, koff[i], blk * (32 * DK * 2));
  };
  auto fetch_v = [&](int blk, int buf) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < kLv; ++i)
      load_row_to_lds(rv, tiles + buf * SH::kTile + 32 * DK + (wg + WPW * i) * 512, voff[i], blk * (32 * DV * 2));
  };
  auto fetch = [&](int blk, int buf) __attribute__((always_inline)) {
    fetch_k(blk, buf);
    fetch_v(blk, buf);
  };
  // all but the youngest n loads have arrived
  auto wait_loads = [&](auto nc) __attribute__((always_inline)) {
    constexpr int n = decltype(nc)::value;
    __builtin_amdgcn_sched_barrier(0);
    __builtin_amdgcn_s_waitcnt(0x0F70 | (n & 15) | ((n >> 4) << 14));
    __builtin_amdgcn_sched_barrier(0);
  };
  const uint8_t* mrow = a.input_mask + (size_t)seq * a.buf_len;
  auto mask_byte = [&](int blk) __attribute__((always_inline)) { return mrow[min(blk * 32 + qi, a.buf_len - 1)]; };
  auto mask_bits = [&](uint8_t mb, int blk) __attribute__((always_inline)) {
    return (uint32_t)__ballot(mb != 0 && blk * 32 + qi < a.buf_len);  // (both halves of the wave say the same)
  };

  const int step0 = max(min(*a.step, min(a.C, a.buf_len) - a.tpp), 0);  // clamped: every slot read lies in the cache
  const int2* place = a.place + (size_t)seq * a.tpp;
  const int first = place[tok].x;                             // oldest slot this query sees (it does not decrease along the tokens)
  const int b_beg = place[q0 / G].x >> 5;                     // blocks of the workgroup
  const int b_end = (step0 + (min(q0 + 32 * SH::WQ, rows) - 1) / G + 32) >> 5;
  const int b_new = step0 >> 5;                               // ROWS: the block of the new row
  uint16_t* const stage = reinterpret_cast<uint16_t*>(ha_smem + SH::kStage);
  int blk = b_beg + split * SH::WP + wp;                      // the block this wave begins with
  uint8_t mb = 0;
  u32x4_t qf[KS];
  if constexpr (ROWS) {
    const HeadLane<KT> hl(ra, lane, min(place[0].y, ra.max_positions - 1));
    const uint16_t* z = reinterpret_cast<const uint16_t*>(ra.z) + (size_t)seq * ra.ldz;
    const bool owner = ((b_new - b_beg) / SH::WP) % a.nsplit == split;  // this workgroup walks the new row's block
    // key (item 0), value (1), then the group's queries, dealt out to the waves, two at a time
    auto items = [&](int i0, auto behind_loads) __attribute__((always_inline)) {
      typename HeadLane<KT>::Head d[2];
      typedef uint16_t val_t __attribute__((ext_vector_type(VT)));
      const bool two = i0 + 4 < G + 2, key = i0 == 0;
      // (all of it is loaded by every wave; items past the last query repeat it)
      const val_t val = *reinterpret_cast<const val_t*>(z + (size_t)(a.H + a.Kh) * DK + (size_t)kvh * DV + VT * lane);
      hl.load(d[0], z + (size_t)(key ? a.H + kvh : kvh * G + max(min(i0 - 2, G - 1), 0)) * DK, key ? ra.k_norm_w : ra.q_norm_w);
      hl.load(d[1], z + (size_t)(kvh * G + min(i0 + 2, G - 1)) * DK, ra.q_norm_w);
      behind_loads();
      if (i0 == 1) {
        *reinterpret_cast<val_t*>(stage + 33 * DK + VT * lane) = val;
        if (owner) *reinterpret_cast<val_t*>(reinterpret_cast<uint16_t*>(ra.vcache) + ((size_t)pair * a.C + step0) * DV + VT * lane) = val;
      } else if (i0 < G + 2) {
        hl.finish(d[0], key ? ra.k_norm_w : ra.q_norm_w, ra.dim, ra.eps);
        store_e<KT>(stage + (key ? 32 : i0 - 2) * DK + hl.c, d[0].v);
        if (key && owner) store_e<KT>(reinterpret_cast<uint16_t*>(ra.kcache) + ((size_t)pair * a.C + step0) * DK + hl.c, d[0].v);
      }
      if (two) {
        hl.finish(d[1], ra.q_norm_w, ra.dim, ra.eps);
        store_e<KT>(stage + (i0 + 2) * DK + hl.c, d[1].v);
      }
    };
    mb = mask_byte(blk);
    items(wave, [&]() __attribute__((always_inline)) {
      if (blk < b_end) fetch(blk, 0);
    });
    for (int i0 = wave + 8; i0 < G + 2; i0 += 8) items(i0, [] {});
    // (the tile under way and the stores of the new row need not be waited for)
    asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
#pragma unroll
    for (int t = 0; t < KS; ++t) qf[t] = *reinterpret_cast<const u32x4_t*>(stage + qr_l * DK + (DK / 2) * h + 8 * t);
  } else {
    const uint16_t* qp = reinterpret_cast<const uint16_t*>(a.q) + qrow * DK + (DK / 2) * h;
#pragma unroll
    for (int t = 0; t < KS; ++t) qf[t] = *reinterpret_cast<const u32x4_t*>(qp + 8 * t);
  }
  const int limit = step0 + tok;                              // newest slot this query sees
  const int limit0 = step0 + min(q0 + wq * 32, rows - 1) / G;  // the smallest one in the wave
  const int first1 = __shfl(first, 31, 64);                   // the largest one in the wave

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
  // behind_scores runs when the block's K rows have been read, v_ready in front of the first read of its V rows
  constexpr bool kLateV = !SHARED && SH::kBufs == 1;
  auto block = [&](int blk, uint32_t mbits, int buf, auto behind_scores, auto v_ready) __attribute__((always_inline)) {
    const uint16_t* kt = tiles + buf * SH::kTile;
    const uint32_t vb = lds_addr(kt) + vbase;
    f32x16_t sacc;
    float mn;
    u32x4_t p[4];  // probabilities as bf16 hi (p[0], p[1]) and lo (p[2], p[3]), 16 positions each
    auto request_v = [&]() __attribute__((always_inline)) {
      static_for<R>([&](auto fc) __attribute__((always_inline)) { load_v(vb, fc); });
      __builtin_amdgcn_sched_barrier(0);
    };
    scores(kt, blk, mbits, sacc, mn);
    behind_scores();
    if (!kLateV) request_v();  // they do not wait for the softmax
    move_reference(mn);
#pragma unroll
    for (int r = 0; r < 16; r += 2) {
      const float p0 = __builtin_amdgcn_exp2f(sacc[r] - m), p1 = __builtin_amdgcn_exp2f(sacc[r + 1] - m);
      const uint32_t hi = pack_bf2(p0, p1);
      p[r >> 3][(r >> 1) & 3] = hi;
      p[2 + (r >> 3)][(r >> 1) & 3] = pack_bf2(p0 - bf_lo(hi), p1 - bf_hi(hi));
      l += p0 + p1;
    }
    if (kLateV) {
      v_ready();
      request_v();
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
    const int rounds = b_end > blk ? (b_end - blk + a.nsplit - 1) / a.nsplit : 0;  // the same in every wave
    mb = mask_byte(blk);
    if (rounds > 0) fetch(blk, 0);
    for (int round = 0; round < rounds; ++round, blk += a.nsplit) {
      const int buf = round & 1;
      const uint32_t mbits = mask_bits(mb, blk);
      __builtin_amdgcn_s_waitcnt(0x0F70);  // this round's tile has landed
      __syncthreads();                     // ... in every wave, and the other buffer's readers are done
      mb = mask_byte(blk + a.nsplit);
      if (round + 1 < rounds) fetch(blk + a.nsplit, buf ^ 1);
      block(blk, mbits, buf, [] {}, [] {});
    }
  } else {
    const int stride = a.nsplit * SH::WP;
    int buf = 0;
    if constexpr (!ROWS) {
      mb = mask_byte(blk);
      if (blk < b_end) fetch(blk, 0);
    }
    uint32_t mbits = mask_bits(mb, blk);
    for (; blk < b_end; blk += stride) {
      const bool more = blk + stride < b_end;
      const bool made = ROWS && blk == b_new;  // the block of the row that waits in LDS
      if (SH::kBufs == 2) mbits = mask_bits(mb, blk);
      // two buffers: the tile has landed; one: its K rows have, the V rows behind them follow
      if (SH::kBufs == 2 || made) wait_loads(IC<0>{});
      else wait_loads(IC<kLv>{});
      if (made) {
        uint16_t* kt = tiles + buf * SH::kTile;
        const int r = step0 & 31;
        if (lane < CK)
          *reinterpret_cast<u32x4_t*>(kt + r * DK + ((lane ^ head_swz<CK>(r)) << 3)) = *reinterpret_cast<const u32x4_t*>(stage + 32 * DK + lane * 8);
        if (lane < CV)
          *reinterpret_cast<u32x4_t*>(kt + 32 * DK + r * DV + ((lane ^ head_swz<CV>(r)) << 3)) =
              *reinterpret_cast<const u32x4_t*>(stage + 33 * DK + lane * 8);
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
      }
      if (SH::kBufs == 2) {
        mb = mask_byte(blk + stride);
        if (more) fetch(blk + stride, buf ^ 1);
        block(blk, mbits, buf, [] {}, [] {});
        buf ^= 1;
      } else {
        // the next K rows travel beside the softmax and the product, the next V rows beside the next scores
        block(blk, mbits, 0,
              [&]() __attribute__((always_inline)) {
                asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
                mb = mask_byte(blk + stride);
                if (more) fetch_k(blk + stride, 0);
              },
              [&]() __attribute__((always_inline)) {
                if (more) {
                  wait_loads(IC<kLk>{});
                  mbits = mask_bits(mb, blk + stride);  // (older than the next K rows)
                } else {
                  wait_loads(IC<0>{});
                }
              });
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        if (more) fetch_v(blk + stride, 0);
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
  const int limit = step0 + row % a.tpp, first = a.place[row].x;
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

int row_places(hipStream_t st, const RowPlacesArgs& a, int M) {
  if (M <= 0 || a.tpp <= 0 || a.buf_len <= 0 || a.C <= 0) return TMX_ERR_SHAPE;
  hipLaunchKernelGGL(row_places_kernel, dim3((M + 255) / 256), dim3(256), 0, st, a, M);
  return check_launch();
}

static bool head_rows_ok(const HeadRowsArgs& a) {
  return a.H > 0 && a.Kh > 0 && a.H % a.Kh == 0 && a.dim > 0 && a.dim <= a.dk && a.rot >= 0 && a.rot % 2 == 0 && a.rot <= a.dim &&
         a.C > 0 && a.buf_len > 0 && a.max_positions > 0 && head_attn_ok(a.dk, a.dv) && a.ldz % 4 == 0 &&
         a.ldz >= (a.H + a.Kh) * a.dk + a.Kh * a.dv;
}

template <typename T>
static int launch_head_rows(hipStream_t st, const HeadRowsArgs& a, int M) {
  const long wgs = (long)M * ((a.H + 2 * a.Kh + 15) / 16);
  if (wgs > 0x7FFFFFFF) return TMX_ERR_SHAPE;
  switch (a.dk) {
    case 64: hipLaunchKernelGGL((head_rows_kernel<T, 1>), dim3(wgs), dim3(256), 0, st, a); break;
    case 128: hipLaunchKernelGGL((head_rows_kernel<T, 2>), dim3(wgs), dim3(256), 0, st, a); break;
    default: hipLaunchKernelGGL((head_rows_kernel<T, 4>), dim3(wgs), dim3(256), 0, st, a); break;
  }
  return check_launch();
}

int head_rows(hipStream_t st, int act, const HeadRowsArgs& a, int M) {
  if (M <= 0 || !head_rows_ok(a)) return TMX_ERR_SHAPE;
  if (act == TMX_ACT_BF16) return launch_head_rows<uint16_t>(st, a, M);
  return act == TMX_ACT_F32 ? launch_head_rows<float>(st, a, M) : TMX_ERR_ARG;
}

// A workgroup holds 128 query rows of a (sequence, kv head), or up to 32 with its waves on different blocks; the slots a
// row sees are split until the CUs are full, as long as a split keeps its waves busy for a while.
struct HeadPlan { bool shared; int nsplit; };
constexpr int kHeadWgs = 512, kHeadMaxSplits = 32, kHeadSplitSlots = 128;
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

template <int KT, int VT, bool SHARED, bool ROWS>
static int launch_head(hipStream_t st, const HeadAttnArgs& a, const HeadRowsArgs& r) {
  using L = HeadShape<KT, VT, SHARED, ROWS>;
  static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(&head_attn_kernel<KT, VT, SHARED, ROWS>),
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, (int)L::kBytes);
  if (attr != hipSuccess) return TMX_ERR_LAUNCH;
  const int rows = a.tpp * (a.H / a.Kh), per = 32 * L::WQ;
  hipLaunchKernelGGL((head_attn_kernel<KT, VT, SHARED, ROWS>), dim3((size_t)a.n_seq * a.Kh * ((rows + per - 1) / per), 1, a.nsplit),
                     dim3(256), L::kBytes, st, a, r);
  return check_launch();
}
template <int KT, int VT>
static int launch_head_kv(hipStream_t st, const HeadAttnArgs& a, bool shared, const HeadRowsArgs* r) {
  if (r) return launch_head<KT, VT, false, true>(st, a, *r);
  return shared ? launch_head<KT, VT, true, false>(st, a, HeadRowsArgs()) : launch_head<KT, VT, false, false>(st, a, HeadRowsArgs());
}
template <int KT>
static int launch_head_v(hipStream_t st, const HeadAttnArgs& a, bool shared, const HeadRowsArgs* r) {
  switch (a.dv) {
    case 64: return launch_head_kv<KT, 1>(st, a, shared, r);
    case 128: return launch_head_kv<KT, 2>(st, a, shared, r);
    default: return launch_head_kv<KT, 4>(st, a, shared, r);
  }
}

bool head_rows_fused(int act, int T, int H, int Kh) { return act == TMX_ACT_BF16 && T == 1 && H / Kh <= 32; }

int head_attention(hipStream_t st, int act, HeadAttnArgs a, const HeadRowsArgs* r) {
  if (a.n_seq <= 0 || a.tpp <= 0 || a.H <= 0 || a.Kh <= 0 || a.H % a.Kh || a.C <= 0 || a.tpp > a.C || a.tpp > a.buf_len ||
      a.chunk < 0 || !head_attn_ok(a.dk, a.dv) || (long)a.n_seq * a.tpp * a.H > 0x3FFFFFFF)
    return TMX_ERR_SHAPE;
  if (r && (!head_rows_fused(act, a.tpp, a.H, a.Kh) || !head_rows_ok(*r) || r->H != a.H || r->Kh != a.Kh || r->dk != a.dk ||
            r->dv != a.dv || r->C != a.C || r->buf_len != a.buf_len))
    return TMX_ERR_ARG;
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
    case 64: rc = launch_head_v<1>(st, a, p.shared, r); break;
    case 128: rc = launch_head_v<2>(st, a, p.shared, r); break;
    default: rc = launch_head_v<4>(st, a, p.shared, r); break;
  }
  if (rc != TMX_OK || a.nsplit == 1) return rc;
  const int total = a.n_seq * a.tpp * a.H;
  hipLaunchKernelGGL(head_combine_kernel, dim3((total + 3) / 4), dim3(256), 0, st, a, total);
  return check_launch();
}

}  // namespace tmx

using namespace tmx;

extern "C" int tmx_row_places(void* stream, const int32_t* positions, const uint8_t* input_mask, const int32_t* step,
                              int buf_len, int32_t* place, int M, int T, int C, int chunk) {
  if (!positions || !input_mask || !step || !place) return TMX_ERR_ARG;
  if (T <= 0 || M % T || chunk < 0) return TMX_ERR_SHAPE;
  RowPlacesArgs a = {};
  a.positions = positions; a.input_mask = input_mask; a.step = step; a.buf_len = buf_len; a.tpp = T; a.C = C; a.chunk = chunk;
  a.place = (int2*)place;
  return row_places((hipStream_t)stream, a, M);
}

static int head_rows_args(HeadRowsArgs& a, const void* z, int ldz, const float* q_norm_w, const float* k_norm_w, float eps,
                          const float* table, int positions_max, const int32_t* place, const int32_t* step, int buf_len,
                          void* q, void* kcache, void* vcache, int T, int H, int Kh, int dim, int dk, int dv, int rot, int C) {
  if (!z || !place || !step || !kcache || !vcache || (rot > 0 && !table)) return TMX_ERR_ARG;
  a.z = z; a.ldz = ldz; a.q_norm_w = q_norm_w; a.k_norm_w = k_norm_w; a.eps = eps;
  a.table = table; a.max_positions = positions_max; a.place = (const int2*)place; a.step = step;
  a.buf_len = buf_len; a.tpp = T; a.q = q; a.kcache = kcache; a.vcache = vcache;
  a.H = H; a.Kh = Kh; a.dim = dim; a.dk = dk; a.dv = dv; a.rot = rot; a.C = C;
  return TMX_OK;
}

extern "C" int tmx_head_rows(void* stream, int act, const void* z, int ldz, const float* q_norm_w, const float* k_norm_w,
                             float eps, const float* table, int positions_max, const int32_t* place,
                             const int32_t* step, int buf_len, void* q, void* kcache, void* vcache, int M, int T, int H,
                             int Kh, int dim, int dk, int dv, int rot, int C) {
  HeadRowsArgs a = {};
  if (!q || head_rows_args(a, z, ldz, q_norm_w, k_norm_w, eps, table, positions_max, place, step, buf_len, q, kcache, vcache,
                           T, H, Kh, dim, dk, dv, rot, C))
    return TMX_ERR_ARG;
  if (T <= 0 || M % T) return TMX_ERR_SHAPE;
  return head_rows((hipStream_t)stream, act, a, M);
}

extern "C" size_t tmx_head_attention_workspace_bytes(int n_seq, int T, int H, int Kh, int dv, int C, int chunk) {
  if (n_seq <= 0 || T <= 0 || H <= 0 || Kh <= 0 || H % Kh || C <= 0) return 0;
  const HeadPlan p = head_plan(n_seq, T, H, Kh, C, chunk);
  return p.nsplit == 1 ? 0 : (size_t)n_seq * T * H * p.nsplit * (dv + 4) * 4;
}

extern "C" int tmx_head_attention(void* stream, int act, const void* q, const void* kcache, const void* vcache,
                                  const float* sink, const int32_t* place, const uint8_t* input_mask, const int32_t* step,
                                  int buf_len, void* out, void* workspace, int n_seq, int T, int H, int Kh, int dk, int dv,
                                  int C, int chunk, float scale) {
  if (!q || !kcache || !vcache || !place || !input_mask || !step || !out) return TMX_ERR_ARG;
  HeadAttnArgs a = {};
  a.q = q; a.kcache = kcache; a.vcache = vcache; a.sink = sink; a.place = (const int2*)place; a.input_mask = input_mask; a.step = step;
  a.buf_len = buf_len; a.out = out; a.partial = (float*)workspace; a.n_seq = n_seq; a.tpp = T; a.H = H; a.Kh = Kh;
  a.dk = dk; a.dv = dv; a.C = C; a.chunk = chunk; a.scale = scale;
  return head_attention((hipStream_t)stream, act, a, nullptr);
}

extern "C" int tmx_head_decode(void* stream, const void* z, int ldz, const float* q_norm_w, const float* k_norm_w, float eps,
                               const float* table, int positions_max, const int32_t* place, void* kcache, void* vcache,
                               const float* sink, const uint8_t* input_mask, const int32_t* step, int buf_len,
                               void* out, void* workspace, int n_seq, int H, int Kh, int dim, int dk, int dv,
                               int rot, int C, int chunk, float scale) {
  HeadRowsArgs r = {};
  if (!input_mask || !out || head_rows_args(r, z, ldz, q_norm_w, k_norm_w, eps, table, positions_max, place, step,
                                                      buf_len, nullptr, kcache, vcache, 1, H, Kh, dim, dk, dv, rot, C))
    return TMX_ERR_ARG;
  HeadAttnArgs a = {};
  a.kcache = kcache; a.vcache = vcache; a.sink = sink; a.place = (const int2*)place; a.input_mask = input_mask; a.step = step;
  a.buf_len = buf_len; a.out = out; a.partial = (float*)workspace; a.n_seq = n_seq; a.tpp = 1; a.H = H; a.Kh = Kh;
  a.dk = dk; a.dv = dv; a.C = C; a.chunk = chunk; a.scale = scale;
  return head_attention((hipStream_t)stream, TMX_ACT_BF16, a, &r);
}
