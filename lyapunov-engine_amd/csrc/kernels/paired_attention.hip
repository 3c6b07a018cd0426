// Differential attention over the paged cache, on the matrix cores, compiled for
// one size of key (LYP_KEY_DIM) and one of value (LYP_VALUE_DIM), multiples of 16.
//
// Every query head has two maps: two queries against two keys of its key/value
// head, each with a softmax of its own over the same visible keys, and both over
// the same values.  With a1 and a2 the two weighted sums of a head,
//     o = a1 - lambda * a2,   o <- o / sqrt(mean(o^2) + eps) * post,   o <- o * sigmoid(gate)
// is what leaves the kernel (no gate given: not gated): a1 and a2 stay in 32-bit registers.
//
// A token at position p sees the keys [first_seen(p), p]: all before it, those of
// a window (p - window, p], or those of its own chunk, the run of `chunk`
// positions counted from 0 that p lies in.
//
//   * paired_prefill: a workgroup takes up to 64 new tokens of one request and up to four query
//     heads of one key/value head (a wave: one head, 16 tokens, both maps).  Key and value tiles pass
//     through two LDS buffers, shared by the four waves; a value fragment read from LDS serves both maps.
//     In launches of few workgroups two sets of four waves share a workgroup's keys, tile about.
//   * paired_decode: a wave takes one request's single new token, all query heads of one
//     key/value head (as the 16 columns of the tile), one map, and a share of a partition of the
//     keys; keys and values go from the pages straight to registers.
// With the keys in several partitions (few new tokens over many keys) the partitions' sums are
// merged by paired_merge, which then finishes the heads.
//
// Pages: keys [page][2 * kv head + map][slot][HD], values [page][kv head][VD][slot].  A query row holds the
// heads one after the other, both maps of a head side by side.
//
// The scores are formed transposed (keys x tokens), which leaves every lane with one token's
// weights for four neighbouring keys of each 16, the operand layout of the product with the
// values; bfloat16 takes 32 keys an instruction there, so value tiles keep their keys in the
// order in which a lane reads them (value_column).
#include <algorithm>

#include "common.h"

#ifndef LYP_KEY_DIM
#error "LYP_KEY_DIM and LYP_VALUE_DIM must be defined"
#endif

namespace lyp {

constexpr int HD = LYP_KEY_DIM;
constexpr int VD = LYP_VALUE_DIM;
static_assert(HD % 16 == 0 && HD >= 16 && HD <= 128 && VD % 16 == 0 && VD >= 16 && VD <= 256, "head sizes in multiples of 16");
constexpr int kMaps = 2;
constexpr int kValueBlocks = VD / 16;
constexpr float kLog2e = 1.4426950408889634f;

__device__ __forceinline__ float fast_exp2(float x) { return __builtin_amdgcn_exp2f(x); }

__device__ __forceinline__ int first_seen(int pos, int window, int chunk) {
  return window > 0 ? max(0, pos - window + 1) : (chunk > 0 ? pos - pos % chunk : 0);
}

__device__ __forceinline__ float lane_groups_max(float v) {
  v = fmaxf(v, __shfl_xor(v, 16, kWave));
  return fmaxf(v, __shfl_xor(v, 32, kWave));
}
__device__ __forceinline__ float lane_groups_sum(float v) {
  v += __shfl_xor(v, 16, kWave);
  return v + __shfl_xor(v, 32, kWave);
}

// How two sums become a head's output.
struct Finish {
  float lambda, eps, post;
  const float* gate;   // [token][gate_ld], the head's VD values at head * VD; null: no gate
  int gate_ld;
};

__device__ __forceinline__ float gated(float o, float g) { return o / (1.0f + expf(-g)); }

template <typename T>
struct Operands {
  using MW = Mma16Wide<T>;
  using WFrag = typename MW::Frag;
  using M4 = Mma16<T>;
  using Frag = typename M4::Frag;
  static constexpr int KE = MW::kElems;             // inner values a lane holds: 8 (bfloat16) or 4 (float)
  static constexpr int KCH = 4 * KE;                // inner values an instruction takes: 32 or 16
  static constexpr int NS = KE / 4;                 // 16-key blocks a step of the sums takes: 2 or 1
  static constexpr int NCW = HD / KCH;              // full steps over the key dimension
  static constexpr bool TAIL = HD % KCH != 0;       // and 16 more values (bfloat16, HD = 32 n + 16)
};

// One map's query (or one key) of a lane: the wide pieces and, where HD asks for it, the last 16 values.
template <typename T>
struct RowFrag {
  using O = Operands<T>;
  typename O::WFrag w[O::NCW > 0 ? O::NCW : 1];
  typename O::Frag tail;
  __device__ __forceinline__ void zero() {
#pragma unroll
    for (int c = 0; c < O::NCW; ++c)
#pragma unroll
      for (int e = 0; e < O::KE; ++e) w[c][e] = from_f32<T>(0.f);
#pragma unroll
    for (int e = 0; e < 4; ++e) tail[e] = from_f32<T>(0.f);
  }
  __device__ __forceinline__ void load(const T* p, int grp) {
#pragma unroll
    for (int c = 0; c < O::NCW; ++c) w[c] = *reinterpret_cast<const typename O::WFrag*>(p + c * O::KCH + O::KE * grp);
    if constexpr (O::TAIL) tail = *reinterpret_cast<const typename O::Frag*>(p + O::NCW * O::KCH + 4 * grp);
  }
};

// Scores of 16 keys (rows) against 16 columns.
template <typename T>
__device__ __forceinline__ f32x4 score(const RowFrag<T>& k, const RowFrag<T>& q) {
  using O = Operands<T>;
  f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int c = 0; c < O::NCW; ++c) s = O::MW::mma(k.w[c], q.w[c], s);
  if constexpr (O::TAIL) {   // a product of its own, added afterwards
    const f32x4 t = O::M4::mma(k.tail, q.tail, f32x4{0.f, 0.f, 0.f, 0.f});
#pragma unroll
    for (int e = 0; e < 4; ++e) s[e] += t[e];
  }
  return s;
}

// The running softmax of one map for one column a lane: maximum in the base-2 domain (the same in
// the four lane groups); `sum` holds the weights' sum in every row (the matrix unit adds them up
// with a row of ones, from the weights as the values' product sees them).
struct Running {
  float m = LYP_NEG_INF;
  f32x4 sum = f32x4{0.f, 0.f, 0.f, 0.f};
};

// The scores of NB 16-key blocks from key kb0 on (s[u]: rows = keys kb0 + 16 u + 4 (lane / 16) + e) become
// weights; the sums so far are rescaled where a maximum grew.  A column sees keys [lo, pos]; MASKED
// false: all of these.
template <typename T, int NB, bool MASKED>
__device__ __forceinline__ void weigh(const f32x4 (&s)[NB], typename Operands<T>::WFrag (&p)[NB / Operands<T>::NS],
                                      float scale_log2, int kb0, int lo, int pos, Running& run, f32x4 (&o)[kValueBlocks],
                                      int grp) {
  constexpr int NS = Operands<T>::NS;
  float mx = LYP_NEG_INF;
  bool vis[NB][4];
#pragma unroll
  for (int u = 0; u < NB; ++u)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      if constexpr (MASKED) {
        const int key = kb0 + 16 * u + 4 * grp + e;
        vis[u][e] = key >= lo && key <= pos;
        mx = fmaxf(mx, vis[u][e] ? s[u][e] : LYP_NEG_INF);
      } else {
        mx = fmaxf(mx, s[u][e]);
      }
    }
  mx = lane_groups_max(mx);
  const float m_new = fmaxf(run.m, mx * scale_log2);   // the scale is positive
  if (__builtin_amdgcn_ballot_w64(m_new > run.m) != 0) {
    const float alpha = fast_exp2(run.m - (m_new == LYP_NEG_INF ? 0.f : m_new));   // 0 while nothing was seen
    run.m = m_new;
#pragma unroll
    for (int e = 0; e < 4; ++e) run.sum[e] *= alpha;
#pragma unroll
    for (int db = 0; db < kValueBlocks; ++db)
#pragma unroll
      for (int e = 0; e < 4; ++e) o[db][e] *= alpha;
  }
  const float m_safe = run.m == LYP_NEG_INF ? 0.f : run.m;
#pragma unroll
  for (int u = 0; u < NB; ++u)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      float w = fast_exp2(__builtin_fmaf(s[u][e], scale_log2, -m_safe));
      if constexpr (MASKED) w = vis[u][e] ? w : 0.f;
      p[u / NS][4 * (u % NS) + e] = from_f32<T>(w);
    }
}

// A finished head of one column: o1, o2 the two maps' sums (lane: values 16 db + 4 grp + e), already divided.
template <typename T>
__device__ __forceinline__ void finish_column(const f32x4 (&o1)[kValueBlocks], float inv1, const f32x4 (&o2)[kValueBlocks],
                                              float inv2, const Finish& fin, size_t token, int head, T* __restrict__ orow,
                                              bool valid, int grp) {
  const float f2 = fin.lambda * inv2;
  float ss = 0.f;
#pragma unroll
  for (int db = 0; db < kValueBlocks; ++db)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float v = o1[db][e] * inv1 - o2[db][e] * f2;
      ss += v * v;
    }
  ss = lane_groups_sum(ss);
  if (!valid) return;
  const float unit = fin.post / sqrtf(ss / static_cast<float>(VD) + fin.eps);
  const float* gate = fin.gate != nullptr ? fin.gate + token * fin.gate_ld + static_cast<size_t>(head) * VD + 4 * grp : nullptr;
#pragma unroll
  for (int db = 0; db < kValueBlocks; ++db) {
    float g[4] = {0.f, 0.f, 0.f, 0.f};
    if (gate != nullptr)
#pragma unroll
      for (int e = 0; e < 4; ++e) g[e] = gate[16 * db + e];
    typename Operands<T>::Frag f;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float v = (o1[db][e] * inv1 - o2[db][e] * f2) * unit;
      f[e] = from_f32<T>(gate != nullptr ? gated(v, g[e]) : v);
    }
    *reinterpret_cast<typename Operands<T>::Frag*>(orow + 16 * db + 4 * grp) = f;
  }
}

// --------------------------------------------------------------------- prefill
template <typename T>
struct Tile {
  using O = Operands<T>;
  static constexpr int kVec = 16 / sizeof(T);                  // elements of a 16-byte piece
  static constexpr int kKLd = kMaps * HD + kVec;               // a key's row: both maps, and a skew of four banks
  static constexpr size_t bytes(int keys) { return (static_cast<size_t>(keys) * kKLd + static_cast<size_t>(VD) * (keys + kVec)) * sizeof(T); }
  static constexpr int kLeast = 16 * O::NS;
  static constexpr int kKeys = bytes(64) <= 40 * 1024 ? 64 : (bytes(32) <= 40 * 1024 ? 32 : kLeast);
  static constexpr int kVLd = kKeys + kVec;
  static constexpr int kElems = kKeys * kKLd + VD * kVLd;
  static constexpr size_t kBytes = 2 * kElems * sizeof(T);     // two buffers
  static constexpr int kKVecs = kKeys * kMaps * HD / kVec, kVVecs = VD * kKeys / kVec;
  static constexpr int kKPer = (kKVecs + 255) / 256, kVPer = (kVVecs + 255) / 256;
  static_assert(kBytes + 2 * kKeys * sizeof(int) <= 160 * 1024, "two tiles must fit the LDS");
  static constexpr bool kMaySplit = sizeof(T) == 2 && 2 * (kBytes + 2 * kKeys * sizeof(int)) <= 160 * 1024 && VD <= 128;
};

// Where a value tile keeps key k: a lane reads its keys of a step (4 of each 16-key block) in one piece.
template <typename T>
__device__ __forceinline__ constexpr int value_column(int k) {
  constexpr int NS = Operands<T>::NS;
  return k / (16 * NS) * (16 * NS) + k % 16 / 4 * (4 * NS) + k / 16 % NS * 4 + k % 4;
}

// KS = 2: two sets of four waves take the workgroup's tiles in turn, each through LDS buffers of its own,
// and the second hands its sums to the first at the end: half as many tiles in a row, for launches whose
// time is that of the workgroup with most keys.
template <typename T, int GH, int KS>
__global__ __launch_bounds__(256 * KS, (HD <= 64 && VD <= 128 && sizeof(T) == 2) ? 2 / KS : 1) void paired_prefill_kernel(
    const T* __restrict__ q, int q_stride, T* __restrict__ out, int out_stride, const T* __restrict__ kpool,
    const T* __restrict__ vpool, const int32_t* __restrict__ block_tables, int table_width,
    const int32_t* __restrict__ q_start, const int32_t* __restrict__ ctx_len, const int32_t* __restrict__ tile_seq,
    const int32_t* __restrict__ tile_q0, int n_tiles, int H, int G, int bs, int page_shift, int window, int chunk,
    float scale_log2, Finish fin, float* __restrict__ part_o, float* __restrict__ part_ml, int n_parts) {
  using TL = Tile<T>;
  using O = Operands<T>;
  constexpr int KT = TL::kKeys, NB = KT / 16, NS = O::NS, NSTEP = NB / NS, VEC = TL::kVec;
  constexpr int QW = (4 / GH) * 16;       // new tokens per workgroup
  constexpr int kSubs = 64 / QW;          // workgroups per 64-token tile of the host's list
  typedef T VecT __attribute__((ext_vector_type(VEC)));
  constexpr int STRIDE = KS * KT;         // from one tile of a set to its next
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  __shared__ int s_page_all[KS][2][KT];
  const int set = KS == 1 ? 0 : __builtin_amdgcn_readfirstlane(static_cast<int>(threadIdx.x) / 256);
  int(*s_page)[KT] = s_page_all[set];
  T* lds = reinterpret_cast<T*>(smem) + set * 2 * TL::kElems;

  const int tid = threadIdx.x % 256, lane = tid % kWave;
  const int wave = __builtin_amdgcn_readfirstlane(tid / kWave);
  const int col = lane % 16, grp = lane / 16;
  const int g = H / G;
  const int head_groups = (g + GH - 1) / GH;
  const int kvh = blockIdx.x / head_groups;
  const int in_group = (blockIdx.x % head_groups) * GH + wave % GH;
  const int head = kvh * g + min(in_group, g - 1);

  // the host lists tiles in rising order of the keys they see; the longest are started first
  const int tile = n_tiles - 1 - static_cast<int>(blockIdx.y) / kSubs;
  const int seq = tile_seq[tile];
  const int tok0 = q_start[seq];
  const int q_len = q_start[seq + 1] - tok0;
  const int ctx = ctx_len[seq];
  const int q0_wg = tile_q0[tile] + (static_cast<int>(blockIdx.y) % kSubs) * QW;
  if (q0_wg >= q_len) return;             // the whole workgroup
  const int pos_first = ctx - q_len + q0_wg;
  const int hi_wg = pos_first + min(QW, q_len - q0_wg);
  const int lo_wg = first_seen(pos_first, window, chunk);

  // this wave's tokens
  const int q0_w = q0_wg + (wave / GH) * 16;
  const bool active = in_group < g && q0_w < q_len;
  const bool valid = active && q0_w + col < q_len;
  const int pos0 = ctx - q_len + q0_w;
  const int pos = pos0 + col, lo = first_seen(pos, window, chunk);
  const int pos_last_w = min(hi_wg - 1, pos0 + 15);
  const int lo_first_w = first_seen(pos0, window, chunk), lo_last_w = first_seen(pos0 + 15, window, chunk);

  RowFrag<T> qf[kMaps];
  const size_t token = static_cast<size_t>(tok0) + q0_w + col;
#pragma unroll
  for (int mp = 0; mp < kMaps; ++mp) {
    qf[mp].zero();
    if (valid) qf[mp].load(q + token * q_stride + static_cast<size_t>(head) * (kMaps * HD) + mp * HD, grp);
  }
  f32x4 o[kMaps][kValueBlocks];
  Running run[kMaps];
#pragma unroll
  for (int mp = 0; mp < kMaps; ++mp)
#pragma unroll
    for (int db = 0; db < kValueBlocks; ++db) o[mp][db] = f32x4{0.f, 0.f, 0.f, 0.f};
  typename O::WFrag ones;
#pragma unroll
  for (int e = 0; e < O::KE; ++e) ones[e] = from_f32<T>(1.f);

  // the tiles of this workgroup: all of its keys, or its run of them
  int k_begin = lo_wg / KT * KT, k_end = hi_wg;
  if (n_parts > 1) {
    const int each = ((hi_wg - k_begin + KT - 1) / KT + n_parts - 1) / n_parts * KT;
    k_begin += static_cast<int>(blockIdx.z) * each;
    k_end = min(hi_wg, k_begin + each);
  }

  const int32_t* table = block_tables + static_cast<size_t>(seq) * table_width;
  auto page_index = [&](int key) { return page_shift >= 0 ? key >> page_shift : key / bs; };
  auto in_page = [&](int key) { return page_shift >= 0 ? key & (bs - 1) : key % bs; };
  // the page of every key of a tile (-1: none), a tile ahead of the loads that need it
  auto locate = [&](int kt0, int buf) {
    if (tid < KT) {
      const int at = page_index(kt0 + tid);
      s_page[buf][tid] = kt0 < k_end && at < table_width ? table[at] : -1;
    }
  };
  VecT kreg[TL::kKPer], vreg[TL::kVPer];
  const bool v_vectors = bs % VEC == 0;
  const size_t k_page_stride = static_cast<size_t>(kMaps * G) * bs * HD, v_page_stride = static_cast<size_t>(G) * VD * bs;
  const T* k_heads = kpool + static_cast<size_t>(kMaps * kvh) * bs * HD;
  const T* v_head = vpool + static_cast<size_t>(kvh) * VD * bs;
  auto zero_vec = [] {
    VecT z;
#pragma unroll
    for (int e = 0; e < VEC; ++e) z[e] = from_f32<T>(0.f);
    return z;
  };
  // Keys outside [lo_wg, hi_wg) become zeros: what their slots hold may be anything.
  auto fetch = [&](int kt0, int buf) {
    const bool inside = kt0 >= lo_wg && kt0 + KT <= hi_wg;
    if (inside && v_vectors) {     // the whole tile exists and is wanted: no tests
#pragma unroll
      for (int n = 0; n < TL::kKPer; ++n) {
        const int piece = min(tid + n * 256, TL::kKVecs - 1);
        const int row = piece / (kMaps * HD / VEC), d = piece % (kMaps * HD / VEC) * VEC;
        kreg[n] = *reinterpret_cast<const VecT*>(k_heads + max(s_page[buf][row], 0) * k_page_stride +
                                                 static_cast<size_t>((d / HD * bs + in_page(kt0 + row)) * HD + d % HD));
      }
#pragma unroll
      for (int n = 0; n < TL::kVPer; ++n) {
        const int piece = min(tid + n * 256, TL::kVVecs - 1);
        const int blk = piece / (VD * (16 / VEC)), d = piece % (VD * (16 / VEC)) / (16 / VEC);
        const int row = 16 * blk + piece % (16 / VEC) * VEC;
        vreg[n] = *reinterpret_cast<const VecT*>(v_head + max(s_page[buf][row], 0) * v_page_stride +
                                                 static_cast<size_t>(d * bs + in_page(kt0 + row)));
      }
      return;
    }
#pragma unroll
    for (int n = 0; n < TL::kKPer; ++n) {
      const int piece = tid + n * 256;
      kreg[n] = zero_vec();
      if (piece >= TL::kKVecs) continue;
      const int row = piece / (kMaps * HD / VEC), d = piece % (kMaps * HD / VEC) * VEC;
      const int key = kt0 + row, page = s_page[buf][row];
      if (page >= 0 && (inside || (key >= lo_wg && key < hi_wg)))
        kreg[n] = *reinterpret_cast<const VecT*>(k_heads + page * k_page_stride +
                                                 static_cast<size_t>((d / HD * bs + in_page(key)) * HD + d % HD));
    }
#pragma unroll
    for (int n = 0; n < TL::kVPer; ++n) {
      const int piece = tid + n * 256;
      vreg[n] = zero_vec();
      if (piece >= TL::kVVecs) continue;
      // 16-key blocks one after the other, inside a block dimension by dimension
      const int blk = piece / (VD * (16 / VEC)), d = piece % (VD * (16 / VEC)) / (16 / VEC);
      const int row = 16 * blk + piece % (16 / VEC) * VEC, key = kt0 + row;
      const T* base = v_head + static_cast<size_t>(d) * bs;
      if (v_vectors) {
        const int page = s_page[buf][row];
        if (page < 0 || key >= hi_wg || key + VEC <= lo_wg) continue;
        vreg[n] = *reinterpret_cast<const VecT*>(base + page * v_page_stride + in_page(key));
        if (!inside)
#pragma unroll
          for (int e = 0; e < VEC; ++e)
            if (key + e < lo_wg || key + e >= hi_wg) vreg[n][e] = from_f32<T>(0.f);
      } else {
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
          const int page = s_page[buf][row + e];
          if (page >= 0 && key + e >= lo_wg && key + e < hi_wg) vreg[n][e] = base[page * v_page_stride + in_page(key + e)];
        }
      }
    }
  };
  auto stash = [&](int buf) {
    T* ks = lds + buf * TL::kElems;
    T* vs = ks + KT * TL::kKLd;
#pragma unroll
    for (int n = 0; n < TL::kKPer; ++n) {
      const int piece = tid + n * 256;
      if (piece >= TL::kKVecs) continue;
      *reinterpret_cast<VecT*>(ks + piece / (kMaps * HD / VEC) * TL::kKLd + piece % (kMaps * HD / VEC) * VEC) = kreg[n];
    }
#pragma unroll
    for (int n = 0; n < TL::kVPer; ++n) {
      const int piece = tid + n * 256;
      if (piece >= TL::kVVecs) continue;
      const int blk = piece / (VD * (16 / VEC)), d = piece % (VD * (16 / VEC)) / (16 / VEC);
      const int row = 16 * blk + piece % (16 / VEC) * VEC;
#pragma unroll
      for (int e = 0; e < VEC; e += 4) {
        typename O::Frag f;
#pragma unroll
        for (int i = 0; i < 4; ++i) f[i] = vreg[n][e + i];
        *reinterpret_cast<typename O::Frag*>(vs + d * TL::kVLd + value_column<T>(row + e)) = f;
      }
    }
  };
  auto compute = [&](int buf, int kt0) __attribute__((always_inline)) {
    const T* ks = lds + buf * TL::kElems;
    const T* vs = ks + KT * TL::kKLd;
    // every token of the wave sees the whole tile: no masks
    const bool full = kt0 + KT - 1 <= pos0 && kt0 >= lo_last_w;
    typename O::WFrag p[kMaps][NSTEP];
#pragma unroll
    for (int mp = 0; mp < kMaps; ++mp) {
      f32x4 s[NB];
#pragma unroll
      for (int u = 0; u < NB; ++u) {
        RowFrag<T> kf;
        kf.load(ks + (16 * u + col) * TL::kKLd + mp * HD, grp);
        s[u] = score<T>(kf, qf[mp]);
      }
      if (full) weigh<T, NB, false>(s, p[mp], scale_log2, kt0, lo, pos, run[mp], o[mp], grp);
      else weigh<T, NB, true>(s, p[mp], scale_log2, kt0, lo, valid ? pos : -1, run[mp], o[mp], grp);
    }
#pragma unroll
    for (int st = 0; st < NSTEP; ++st) {
#pragma unroll
      for (int mp = 0; mp < kMaps; ++mp) run[mp].sum = O::MW::mma(ones, p[mp][st], run[mp].sum);
      const T* vrow = vs + col * TL::kVLd + st * 16 * NS + grp * O::KE;
#pragma unroll
      for (int db = 0; db < kValueBlocks; ++db) {
        const typename O::WFrag vf = *reinterpret_cast<const typename O::WFrag*>(vrow + db * 16 * TL::kVLd);
#pragma unroll
        for (int mp = 0; mp < kMaps; ++mp) o[mp][db] = O::MW::mma(vf, p[mp][st], o[mp][db]);
      }
    }
  };

  if (k_begin < k_end) {     // (a run of a cut unit may be empty: the whole workgroup agrees on it)
    const int first = k_begin + set * KT;
    locate(first, 0);
    locate(first + STRIDE, 1);
    __syncthreads();
    if (first < k_end) {
      fetch(first, 0);
      stash(0);
    }
    __syncthreads();
    int buf = 0;
    // the bounds are those of set 0, so that every wave passes the same barriers
    for (int kb = k_begin; kb < k_end; kb += STRIDE, buf ^= 1) {
      const int kt0 = kb + set * KT;
      const bool more = kt0 + STRIDE < k_end;
      if (more) {
        fetch(kt0 + STRIDE, buf ^ 1);
        locate(kt0 + 2 * STRIDE, buf);        // this tile's own entries were used a round ago
      }
      if (active && kt0 < k_end && kt0 <= pos_last_w && kt0 + KT > lo_first_w) compute(buf, kt0);
      if (more) stash(buf ^ 1);
      __syncthreads();
    }
  }

  if constexpr (KS == 2) {
    // set 1 hands maximum, sum and output of both maps to the same wave and lane of set 0, map by map
    constexpr int kHand = 2 + 4 * kValueBlocks;
    static_assert(256 * kHand * sizeof(float) <= KS * TL::kBytes, "the hand-over goes through the tile buffers");
    float* hand = reinterpret_cast<float*>(smem) + tid;
#pragma unroll
    for (int mp = 0; mp < kMaps; ++mp) {
      if (set == 1) {
        hand[0] = run[mp].m;
        hand[256] = run[mp].sum[0];
#pragma unroll
        for (int db = 0; db < kValueBlocks; ++db)
#pragma unroll
          for (int e = 0; e < 4; ++e) hand[(2 + 4 * db + e) * 256] = o[mp][db][e];
      }
      __syncthreads();
      if (set == 0) {
        const float m_other = hand[0], m_new = fmaxf(run[mp].m, m_other);
        const float m_safe = m_new == LYP_NEG_INF ? 0.f : m_new;
        const float a0 = fast_exp2(run[mp].m - m_safe), a1 = fast_exp2(m_other - m_safe);   // 0 for a set that saw nothing
        run[mp].sum[0] = run[mp].sum[0] * a0 + hand[256] * a1;
#pragma unroll
        for (int db = 0; db < kValueBlocks; ++db)
#pragma unroll
          for (int e = 0; e < 4; ++e) o[mp][db][e] = o[mp][db][e] * a0 + hand[(2 + 4 * db + e) * 256] * a1;
        run[mp].m = m_new;
      }
      __syncthreads();
    }
    if (set == 1) return;      // (no barrier follows)
  }

  if (n_parts > 1) {
    if (valid) {
      const int in_tile = q0_w - tile_q0[tile] + col;
#pragma unroll
      for (int mp = 0; mp < kMaps; ++mp) {
        const size_t at = (((static_cast<size_t>(tile) * 64 + in_tile) * H + head) * kMaps + mp) * n_parts + blockIdx.z;
        float* po = part_o + at * VD + 4 * grp;
#pragma unroll
        for (int db = 0; db < kValueBlocks; ++db) *reinterpret_cast<f32x4*>(po + db * 16) = o[mp][db];
        if (grp == 0) {
          part_ml[at * 2] = run[mp].m;
          part_ml[at * 2 + 1] = run[mp].sum[0];
        }
      }
    }
    return;
  }
  const float l1 = run[0].sum[0], l2 = run[1].sum[0];
  finish_column<T>(o[0], l1 > 0.f ? 1.0f / l1 : 0.f, o[1], l2 > 0.f ? 1.0f / l2 : 0.f, fin, token, head,
                   out + token * out_stride + static_cast<size_t>(head) * VD, valid, grp);
}

// ------------------------------------------------------- merging partitions
constexpr int kPartsMost = 128;
constexpr int kMergeThreads = 256;

// A workgroup: the first count() partitions of one token's head (their results at index base + map * most + p),
// put together and finished.  A thread a (map, value); the maxima, weights and denominators a wave a map, a lane
// a partition.
template <typename T, typename Count>
__device__ __forceinline__ void merge_head(const float* __restrict__ part_o, const float* __restrict__ part_ml, size_t base,
                                           int most, Count count, const Finish& fin, size_t token, int head,
                                           T* __restrict__ orow) {
  __shared__ float s_w[kMaps][kPartsMost];
  __shared__ float s_inv[kMaps];
  __shared__ float s_v[kMaps][VD];
  __shared__ float s_ss[kMergeThreads / kWave];
  constexpr int PER = (kMaps * VD + kMergeThreads - 1) / kMergeThreads;
  const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave;
  // The first partitions' results are asked for before anything else is known (one that does not exist holds
  // whatever the workspace held; it is dropped): the kernel is as long as its chain of loads.
  constexpr int kFirst = 4;
  float first[PER][kFirst];
#pragma unroll
  for (int k = 0; k < PER; ++k) {
    const int i = min(tid + k * kMergeThreads, kMaps * VD - 1);
#pragma unroll
    for (int p = 0; p < kFirst; ++p)
      first[k][p] = part_o[(base + static_cast<size_t>(i / VD) * most + min(p, most - 1)) * VD + i % VD];
  }
  const int n = count();
  if (wave < kMaps) {
    const float2* ml = reinterpret_cast<const float2*>(part_ml) + base + static_cast<size_t>(wave) * most;
    constexpr int EACH = kPartsMost / kWave;
    float2 r[EACH];
    float m = LYP_NEG_INF, l = 0.f;
#pragma unroll
    for (int e = 0; e < EACH; ++e) {
      const int p = lane + e * kWave;
      r[e] = p < n ? ml[p] : float2{LYP_NEG_INF, 0.f};
      m = fmaxf(m, r[e].x);
    }
    m = wave_max(m);
    const float m_safe = m == LYP_NEG_INF ? 0.f : m;
#pragma unroll
    for (int e = 0; e < EACH; ++e) {
      const float w = fast_exp2(r[e].x - m_safe);
      l += w * r[e].y;
      s_w[wave][lane + e * kWave] = w;
    }
    l = wave_sum(l);
    if (lane == 0) s_inv[wave] = l > 0.f ? 1.0f / l : 0.f;
  }
  __syncthreads();
#pragma unroll
  for (int k = 0; k < PER; ++k) {
    const int i = tid + k * kMergeThreads;
    if (i >= kMaps * VD) continue;
    const int mp = i / VD, d = i % VD;
    float acc = 0.f;
#pragma unroll
    for (int p = 0; p < kFirst; ++p) acc += p < n ? s_w[mp][p] * first[k][p] : 0.f;
    const float* src = part_o + (base + static_cast<size_t>(mp) * most) * VD + d;
#pragma unroll 8
    for (int p = kFirst; p < n; ++p) acc += s_w[mp][p] * src[static_cast<size_t>(p) * VD];
    s_v[mp][d] = acc * s_inv[mp];
  }
  __syncthreads();
  float o = 0.f;
  if (tid < VD) o = s_v[0][tid] - fin.lambda * s_v[1][tid];
  const float part = wave_sum(o * o);
  if (lane == 0) s_ss[wave] = part;
  __syncthreads();
  if (tid >= VD) return;
  float ss = 0.f;
#pragma unroll
  for (int w = 0; w < kMergeThreads / kWave; ++w) ss += s_ss[w];
  const float y = o * (fin.post / sqrtf(ss / static_cast<float>(VD) + fin.eps));
  orow[tid] = from_f32<T>(fin.gate != nullptr ? gated(y, fin.gate[token * fin.gate_ld + static_cast<size_t>(head) * VD + tid]) : y);
}

// grid (H, 64, tiles): the runs of one new token's head after a cut prefill.
template <typename T>
__global__ __launch_bounds__(kMergeThreads) void paired_merge_prefill_kernel(
    const float* __restrict__ part_o, const float* __restrict__ part_ml, int n_parts, const int32_t* __restrict__ q_start,
    const int32_t* __restrict__ tile_seq, const int32_t* __restrict__ tile_q0, T* __restrict__ out, int out_stride, int H,
    Finish fin) {
  const int head = blockIdx.x, in_tile = blockIdx.y, tile = blockIdx.z;
  const int seq = tile_seq[tile];
  const int tok0 = q_start[seq], q_len = q_start[seq + 1] - tok0;
  const int qi = tile_q0[tile] + in_tile;
  if (qi >= q_len) return;
  const size_t token = static_cast<size_t>(tok0) + qi;
  merge_head<T>(part_o, part_ml, ((static_cast<size_t>(tile) * 64 + in_tile) * H + head) * kMaps * n_parts, n_parts,
                [&] { return n_parts; }, fin, token, head, out + token * out_stride + static_cast<size_t>(head) * VD);
}

// ---------------------------------------------------------------------- decode
// Eight waves a workgroup: wave w takes map w % 2 and share w / 2 of the partition's keys.  (The two waves of a
// share read the same values at the same time, the second from the cache; with both maps in one wave its
// registers would hold half as many keys on their way.)
constexpr int kDecodeWaves = 8;
constexpr int kShares = kDecodeWaves / kMaps;
constexpr int kShareKeys = VD <= 128 ? 64 : 32;     // the smallest share
constexpr int kDecodeLeast = kShares * kShareKeys;  // keys of the smallest partition

// The keys one workgroup takes of the n a request's token sees when a partition may hold `most` of
// them: as many partitions as that needs, of even size, in whole smallest shares.
__device__ __forceinline__ int decode_part_keys(int n, int most) {
  const int parts = max(1, (n + most - 1) / most);
  const int per = (n + parts - 1) / parts;
  return max(kDecodeLeast, (per + kDecodeLeast - 1) / kDecodeLeast * kDecodeLeast);
}

// LDS of a workgroup: every wave's sums of its map for the columns that hold a head, maxima and sums.
constexpr size_t decode_lds_floats(int g) { return static_cast<size_t>(kDecodeWaves) * ((g < 16 ? g : 16) * VD + 32); }

// grid (partitions, G * column groups, requests).  WHOLE: one partition a request, which the workgroup
// finishes by itself.  ALIGNED: pages of a multiple of 16 slots, so that a block of 16 keys lies in one page: its
// address is then the same for the whole wave, and a block is read whole wherever a key of it is wanted (what the
// other slots hold, NaN included, is dropped: scores by their mask, values by clear_unseen).
template <typename T, bool WHOLE, bool ALIGNED>
__global__ __launch_bounds__(kDecodeWaves* kWave) void paired_decode_kernel(
    const T* __restrict__ q, int q_stride, const T* __restrict__ kpool, const T* __restrict__ vpool,
    const int32_t* __restrict__ block_tables, int table_width, const int32_t* __restrict__ q_start,
    const int32_t* __restrict__ ctx_len, const int32_t* __restrict__ dec_seqs, float* __restrict__ part_o,
    float* __restrict__ part_ml, int max_parts, int most_keys, int H, int G, int bs, int page_shift, int window, int chunk,
    float scale_log2, T* __restrict__ out, int out_stride, Finish fin) {
  using O = Operands<T>;
  constexpr int NS = O::NS, STEP = sizeof(T) == 2 ? kShareKeys : (VD <= 128 ? 32 : 16), NB = STEP / 16, NSTEP = NB / NS;   // keys a round
  extern __shared__ float s_dec[];
  const int lane = threadIdx.x % kWave;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWave);
  const int mp = wave % kMaps, share = wave / kMaps;
  const int col = lane % 16, grp = lane / 16;
  const int g = H / G, cols_most = min(16, g);
  float* s_o = s_dec;                                      // [waves][cols_most][VD]
  float* s_m = s_o + kDecodeWaves * cols_most * VD;        // [waves][16]
  float* s_l = s_m + kDecodeWaves * 16;
  const int col_groups = (g + 15) / 16;
  const int kvh = blockIdx.y / col_groups, h0 = (blockIdx.y % col_groups) * 16;
  const int slot = blockIdx.z, seq = dec_seqs != nullptr ? dec_seqs[slot] : slot;
  const int ctx = ctx_len[seq];
  const size_t token = q_start[seq];
  const int pos = ctx - 1, lo = ctx > 0 ? first_seen(pos, window, chunk) : 0;
  const int lo16 = lo / 16 * 16;
  const int part_keys = decode_part_keys(ctx - lo16, most_keys);
  const int part_begin = lo16 + static_cast<int>(blockIdx.x) * part_keys;
  if (!WHOLE && part_begin >= ctx) return;        // the whole workgroup (the merge knows how many there are)
  const int k_begin = part_begin + share * (part_keys / kShares);
  const int k_end = min(ctx, k_begin + part_keys / kShares);

  const bool col_valid = h0 + col < g;
  const int head = kvh * g + h0 + (col_valid ? col : 0);
  RowFrag<T> qf;
  qf.zero();
  if (col_valid) qf.load(q + token * q_stride + static_cast<size_t>(head) * (kMaps * HD) + mp * HD, grp);
  f32x4 o[kValueBlocks];
  Running run;
#pragma unroll
  for (int db = 0; db < kValueBlocks; ++db) o[db] = f32x4{0.f, 0.f, 0.f, 0.f};
  typename O::WFrag ones;
#pragma unroll
  for (int e = 0; e < O::KE; ++e) ones[e] = from_f32<T>(1.f);

  const int32_t* table = block_tables + static_cast<size_t>(seq) * table_width;
  auto page_at = [&](int key) {
    const int at = page_shift >= 0 ? key >> page_shift : key / bs;
    return at < table_width ? table[at] : -1;
  };
  auto in_page = [&](int key) { return page_shift >= 0 ? key & (bs - 1) : key % bs; };
  const T* k_head = kpool + static_cast<size_t>(kMaps * kvh + mp) * bs * HD;
  const T* v_head = vpool + (static_cast<size_t>(kvh) * VD + col) * bs;
  const size_t k_page_stride = static_cast<size_t>(kMaps * G) * bs * HD, v_page_stride = static_cast<size_t>(G) * VD * bs;
  RowFrag<T> kf[NB];
  typename O::WFrag vf[NSTEP][kValueBlocks];
  // pages of the round's keys: this lane's key of every 16-key block (keys), and the first of its four (values)
  int kpage[NB], vpage[NB];
  auto pages_of = [&](int kb0) {
    if constexpr (ALIGNED) {
#pragma unroll
      for (int u = 0; u < NB; ++u)
        kpage[u] = __builtin_amdgcn_readfirstlane(table[min(page_shift >= 0 ? (kb0 + 16 * u) >> page_shift : (kb0 + 16 * u) / bs,
                                                            table_width - 1)]);
      return;
    }
#pragma unroll
    for (int u = 0; u < NB; ++u) {
      kpage[u] = page_at(kb0 + 16 * u + col);
      vpage[u] = page_at(kb0 + 16 * u + 4 * grp);
    }
  };
  auto wanted = [&](int u, int kb0) {     // ALIGNED: whether any key of a block is
    return kb0 + 16 * u < k_end && kb0 + 16 * u + 16 > lo && kpage[u] >= 0;
  };
  auto load_keys = [&](int kb0) {
    if constexpr (ALIGNED) {
#pragma unroll
      for (int u = 0; u < NB; ++u) {
        if (wanted(u, kb0))
          kf[u].load(k_head + kpage[u] * k_page_stride + static_cast<size_t>(in_page(kb0 + 16 * u)) * HD + col * HD, grp);
        else
          kf[u].zero();
      }
      return;
    }
#pragma unroll
    for (int u = 0; u < NB; ++u) {
      const int key = kb0 + 16 * u + col;
      if (key >= lo && key < k_end && kpage[u] >= 0)
        kf[u].load(k_head + kpage[u] * k_page_stride + static_cast<size_t>(in_page(key)) * HD, grp);
      else
        kf[u].zero();
    }
  };
  const bool v_quads = bs % 4 == 0;
  auto load_values = [&](int kb0) {
    if constexpr (ALIGNED) {
#pragma unroll
      for (int u = 0; u < NB; ++u) {
        const bool in = wanted(u, kb0);
        const T* at = vpool + max(kpage[u], 0) * v_page_stride + static_cast<size_t>(kvh) * VD * bs + in_page(kb0 + 16 * u);
        const int mine = col * bs + 4 * grp;
#pragma unroll
        for (int db = 0; db < kValueBlocks; ++db) {
          typename O::Frag f;
          if (in) {
            f = *reinterpret_cast<const typename O::Frag*>(at + db * 16 * bs + mine);
          } else {
#pragma unroll
            for (int e = 0; e < 4; ++e) f[e] = from_f32<T>(0.f);
          }
#pragma unroll
          for (int e = 0; e < 4; ++e) vf[u / NS][db][4 * (u % NS) + e] = f[e];
        }
      }
      return;
    }
#pragma unroll
    for (int u = 0; u < NB; ++u) {
      const int key0 = kb0 + 16 * u + 4 * grp;
      if (v_quads) {
        const bool any = vpage[u] >= 0 && key0 < k_end && key0 + 3 >= lo;
        const T* at = v_head + max(vpage[u], 0) * v_page_stride + in_page(key0);
#pragma unroll
        for (int db = 0; db < kValueBlocks; ++db) {
          typename O::Frag f;
#pragma unroll
          for (int e = 0; e < 4; ++e) f[e] = from_f32<T>(0.f);
          if (any) f = *reinterpret_cast<const typename O::Frag*>(at + db * 16 * bs);
#pragma unroll
          for (int e = 0; e < 4; ++e) vf[u / NS][db][4 * (u % NS) + e] = f[e];
        }
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int key = key0 + e;
          const int page = key >= lo && key < k_end ? page_at(key) : -1;
          const T* at = v_head + max(page, 0) * v_page_stride + in_page(key);
#pragma unroll
          for (int db = 0; db < kValueBlocks; ++db)
            vf[u / NS][db][4 * (u % NS) + e] = page >= 0 ? at[db * 16 * bs] : from_f32<T>(0.f);
        }
      }
    }
  };
  // keys of a quad that nobody sees: whatever their slots hold becomes zero, where a round's edge makes that necessary
  auto clear_unseen = [&](int kb0) {
#pragma unroll
    for (int u = 0; u < NB; ++u)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int key = kb0 + 16 * u + 4 * grp + e;
        if (key >= lo && key < k_end) continue;
#pragma unroll
        for (int db = 0; db < kValueBlocks; ++db) vf[u / NS][db][4 * (u % NS) + e] = from_f32<T>(0.f);
      }
  };
  if (k_begin < k_end) {
    pages_of(k_begin);
    load_keys(k_begin);
    load_values(k_begin);
  }
  for (int kb0 = k_begin; kb0 < k_end; kb0 += STEP) {
    const bool more = kb0 + STEP < k_end;
    if (more) pages_of(kb0 + STEP);
    f32x4 s[NB];
#pragma unroll
    for (int u = 0; u < NB; ++u) s[u] = score<T>(kf[u], qf);
    if (more) load_keys(kb0 + STEP);
    typename O::WFrag p[NSTEP];
    if (kb0 >= lo && kb0 + STEP <= k_end) {
      weigh<T, NB, false>(s, p, scale_log2, kb0, lo, pos, run, o, grp);
    } else {
      weigh<T, NB, true>(s, p, scale_log2, kb0, lo, k_end - 1, run, o, grp);
      clear_unseen(kb0);
    }
#pragma unroll
    for (int st = 0; st < NSTEP; ++st) {
      run.sum = O::MW::mma(ones, p[st], run.sum);
#pragma unroll
      for (int db = 0; db < kValueBlocks; ++db) o[db] = O::MW::mma(vf[st][db], p[st], o[db]);
    }
    if (more) load_values(kb0 + STEP);
  }

  if (col < cols_most) {
#pragma unroll
    for (int db = 0; db < kValueBlocks; ++db)
      *reinterpret_cast<f32x4*>(&s_o[(wave * cols_most + col) * VD + db * 16 + 4 * grp]) = o[db];
  }
  if (lane < 16) {
    s_m[wave * 16 + col] = col_valid ? run.m : LYP_NEG_INF;
    s_l[wave * 16 + col] = run.sum[0];
  }
  __syncthreads();

  // a wave a column: the shares' results of both maps put together, in the order of the shares
  constexpr int PER = (VD + kWave - 1) / kWave;
  const int ncols = min(16, g - h0);
  for (int c = wave; c < ncols; c += kDecodeWaves) {
    const int hh = kvh * g + h0 + c;
    float v[kMaps][PER], inv[kMaps];
#pragma unroll
    for (int m2 = 0; m2 < kMaps; ++m2) {
      float m = LYP_NEG_INF;
#pragma unroll
      for (int w = 0; w < kShares; ++w) m = fmaxf(m, s_m[(w * kMaps + m2) * 16 + c]);
      const float m_safe = m == LYP_NEG_INF ? 0.f : m;
      float l = 0.f;
#pragma unroll
      for (int k = 0; k < PER; ++k) v[m2][k] = 0.f;
#pragma unroll
      for (int w = 0; w < kShares; ++w) {
        const int from = w * kMaps + m2;
        const float wgt = fast_exp2(s_m[from * 16 + c] - m_safe);
        l += wgt * s_l[from * 16 + c];
#pragma unroll
        for (int k = 0; k < PER; ++k) {
          const int d = lane + kWave * k;
          if (d < VD) v[m2][k] += wgt * s_o[(from * cols_most + c) * VD + d];
        }
      }
      if constexpr (!WHOLE) {
        const size_t at = ((static_cast<size_t>(slot) * H + hh) * kMaps + m2) * max_parts + blockIdx.x;
#pragma unroll
        for (int k = 0; k < PER; ++k) {
          const int d = lane + kWave * k;
          if (d < VD) part_o[at * VD + d] = v[m2][k];
        }
        if (lane == 0) {
          part_ml[at * 2] = m;
          part_ml[at * 2 + 1] = l;
        }
      }
      inv[m2] = l > 0.f ? 1.0f / l : 0.f;
    }
    if constexpr (WHOLE) {
      float ss = 0.f;
#pragma unroll
      for (int k = 0; k < PER; ++k) {
        v[0][k] = v[0][k] * inv[0] - fin.lambda * (v[1][k] * inv[1]);
        if (lane + kWave * k < VD) ss += v[0][k] * v[0][k];
      }
      ss = wave_sum(ss);
      const float unit = fin.post / sqrtf(ss / static_cast<float>(VD) + fin.eps);
      const float* gate = fin.gate != nullptr ? fin.gate + token * fin.gate_ld + static_cast<size_t>(hh) * VD : nullptr;
      T* orow = out + token * out_stride + static_cast<size_t>(hh) * VD;
#pragma unroll
      for (int k = 0; k < PER; ++k) {
        const int d = lane + kWave * k;
        if (d >= VD) continue;
        const float y = v[0][k] * unit;
        orow[d] = from_f32<T>(gate != nullptr ? gated(y, gate[d]) : y);
      }
    }
  }
}

// grid (H, requests): the partitions of one request's token and head.
template <typename T>
__global__ __launch_bounds__(kMergeThreads) void paired_merge_decode_kernel(
    const float* __restrict__ part_o, const float* __restrict__ part_ml, int max_parts, int most_keys,
    const int32_t* __restrict__ q_start, const int32_t* __restrict__ ctx_len, const int32_t* __restrict__ dec_seqs,
    T* __restrict__ out, int out_stride, int H, int window, int chunk, Finish fin) {
  const int head = blockIdx.x, slot = blockIdx.y, seq = dec_seqs != nullptr ? dec_seqs[slot] : slot;
  const int ctx = ctx_len[seq];
  const size_t token = q_start[seq];
  auto live = [&] {
    const int lo16 = ctx > 0 ? first_seen(ctx - 1, window, chunk) / 16 * 16 : 0;
    const int part_keys = decode_part_keys(ctx - lo16, most_keys);
    return min(max_parts, (ctx - lo16 + part_keys - 1) / part_keys);
  };
  merge_head<T>(part_o, part_ml, (static_cast<size_t>(slot) * H + head) * kMaps * max_parts, max_parts, live, fin, token, head,
                out + token * out_stride + static_cast<size_t>(head) * VD);
}

constexpr int kPrefillPartsMost = 16;
constexpr int kPartAlone = 256;    // partitions up to this size are merged in pairs where that leaves one

static int shift_of(int bs) {
  if ((bs & (bs - 1)) != 0) return -1;
  int s = 0;
  while ((1 << s) < bs) ++s;
  return s;
}

static int heads_per_workgroup(int g) { return g >= 4 ? 4 : (g >= 2 ? 2 : 1); }

static int check_common(const char* name, int H, int G, int bs, int table_width, int q_stride, int out_stride, int window,
                        int chunk, const void* q, const void* kpool, const void* vpool, const float* gate, int gate_ld) {
  LYP_REQUIRE(H > 0 && G > 0 && H % G == 0, "%s: %d query heads over %d key/value heads", name, H, G);
  LYP_REQUIRE(bs > 0 && table_width > 0, "%s: page size %d, table width %d", name, bs, table_width);
  LYP_REQUIRE(q_stride >= H * kMaps * HD && q_stride % 8 == 0, "%s: query row stride %d", name, q_stride);
  LYP_REQUIRE(out_stride >= H * VD && out_stride % 4 == 0, "%s: output row stride %d", name, out_stride);
  LYP_REQUIRE(window >= 0 && chunk >= 0 && (window == 0 || chunk == 0), "%s: a window of %d and a chunk of %d", name, window, chunk);
  LYP_REQUIRE(reinterpret_cast<uintptr_t>(q) % 16 == 0 && reinterpret_cast<uintptr_t>(kpool) % 16 == 0 &&
                  reinterpret_cast<uintptr_t>(vpool) % 16 == 0, "%s: operands must be 16-byte aligned", name);
  LYP_REQUIRE(gate == nullptr || gate_ld >= H * VD, "%s: gate rows of %d", name, gate_ld);
  return 0;
}

}  // namespace lyp

using namespace lyp;

extern "C" {

int lyp_paired_key_dim() { return HD; }
int lyp_paired_value_dim() { return VD; }

// Keys per workgroup at most for a decode launch over n_seqs requests whose tokens see up to max_keys keys.
int lyp_paired_decode_plan(int n_seqs, int max_keys, int H, int G) {
  auto pow2 = [](int v, int least) {
    int p = least;
    while (p < v) p *= 2;
    return p;
  };
  const int g = H / std::max(G, 1);
  const long long base = static_cast<long long>(pow2(n_seqs, 1)) * G * ((g + 15) / 16);
  int part = kDecodeLeast;
  while ((max_keys + part - 1) / part > kPartsMost) part *= 2;
  // partitions grow while the launch keeps a workgroup per compute unit
  while (part < max_keys && base * ((max_keys + 2 * part - 1) / (2 * part)) >= compute_units()) part *= 2;
  // two short partitions a request are not worth the merge they need
  if (2 * part >= max_keys && part < max_keys && part <= kPartAlone) part *= 2;
  return part;
}

// Into how many runs lyp_paired_prefill had better cut every tile's keys (1: not at all), for n_tiles tiles
// of 64 new tokens of which one sees max_keys keys.  More than one needs a workspace: n_tiles * 64 * H * 2 *
// parts * VD floats for part_o, n_tiles * 64 * H * 2 * parts * 2 for part_ml.
int lyp_paired_prefill_plan(int n_tiles, int max_keys, int H, int G, int dtype) {
  if (n_tiles <= 0 || G <= 0) return 1;
  const int g = H / G, gh = heads_per_workgroup(g);
  const long long wgs = static_cast<long long>(n_tiles) * gh * G * ((g + gh - 1) / gh);   // 4 / gh blocks of 16 tokens each
  const int kt = dtype == kF32 ? Tile<float>::kKeys : Tile<bf16_t>::kKeys;
  const int tiles = (max_keys + kt - 1) / kt;
  int parts = 1;
  while (parts < kPrefillPartsMost && wgs * parts < compute_units() && tiles / (2 * parts) >= 8) parts *= 2;
  return parts;
}

int lyp_paired_prefill(const void* q, int q_stride, void* out, int out_stride, const void* kpool, const void* vpool,
                       int dtype, const int32_t* block_tables, int table_width, const int32_t* q_start,
                       const int32_t* ctx_len, const int32_t* tile_seq, const int32_t* tile_q0, int n_tiles, int H, int G,
                       int bs, int window, int chunk, float scale, float lambda, float eps, float post, const float* gate,
                       int gate_ld, float* part_o, float* part_ml, int n_parts, hipStream_t stream) {
  if (check_common("paired_prefill", H, G, bs, table_width, q_stride, out_stride, window, chunk, q, kpool, vpool, gate, gate_ld))
    return -1;
  LYP_REQUIRE(scale > 0.f, "paired_prefill: a scale of %g", static_cast<double>(scale));
  LYP_REQUIRE(n_tiles >= 0 && n_tiles <= 8191, "paired_prefill: %d tiles in one launch", n_tiles);
  LYP_REQUIRE(n_parts >= 1 && n_parts <= kPrefillPartsMost && (n_parts == 1 || (part_o && part_ml)),
              "paired_prefill: %d runs of the keys (at most %d, with a workspace)", n_parts, kPrefillPartsMost);
  LYP_REQUIRE(dtype == kF32 || dtype == kBF16, "paired_prefill: unknown dtype %d", dtype);
  if (n_tiles == 0) return 0;
  const int g = H / G, gh = heads_per_workgroup(g);
  const Finish fin{lambda, eps, post, gate, gate_ld};
  const dim3 grid(G * ((g + gh - 1) / gh), n_tiles * gh, n_parts);
  const float scale_log2 = scale * kLog2e;
  // Two sets of waves a workgroup while the launch has at most `kSplitBelow` workgroups per compute unit.
  constexpr int kSplitBelow = 2;
  const bool split = static_cast<long long>(grid.x) * grid.y * grid.z <= static_cast<long long>(kSplitBelow) * compute_units();
#define LYP_PAIRED_KS(T, GH, KS)                                                                                       \
  do {                                                                                                                 \
    static bool asked = false;   /* the tiles may take more LDS than a kernel gets unasked */                          \
    if (!asked) {                                                                                                      \
      (void)hipFuncSetAttribute(reinterpret_cast<const void*>(paired_prefill_kernel<T, GH, KS>),                       \
                                hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(KS * Tile<T>::kBytes));   \
      asked = true;                                                                                                    \
    }                                                                                                                  \
    paired_prefill_kernel<T, GH, KS><<<grid, 256 * KS, KS * Tile<T>::kBytes, stream>>>(                                \
        static_cast<const T*>(q), q_stride, static_cast<T*>(out), out_stride, static_cast<const T*>(kpool),            \
        static_cast<const T*>(vpool), block_tables, table_width, q_start, ctx_len, tile_seq, tile_q0, n_tiles, H, G,   \
        bs, shift_of(bs), window, chunk, scale_log2, fin, part_o, part_ml, n_parts);                                   \
  } while (0)
#define LYP_PAIRED(T, GH)                                   \
  do {                                                      \
    if constexpr (Tile<T>::kMaySplit) {                     \
      if (split) {                                          \
        LYP_PAIRED_KS(T, GH, 2);                            \
        break;                                              \
      }                                                     \
    }                                                       \
    LYP_PAIRED_KS(T, GH, 1);                                \
  } while (0)
#define LYP_PAIRED_T(T)                   \
  do {                                    \
    if (gh == 4) LYP_PAIRED(T, 4);        \
    else if (gh == 2) LYP_PAIRED(T, 2);   \
    else LYP_PAIRED(T, 1);                \
    if (n_parts > 1)                      \
      paired_merge_prefill_kernel<T><<<dim3(H, 64, n_tiles), kMergeThreads, 0, stream>>>(            \
          part_o, part_ml, n_parts, q_start, tile_seq, tile_q0, static_cast<T*>(out), out_stride, H, fin); \
  } while (0)
  if (dtype == kF32) LYP_PAIRED_T(float);
  else LYP_PAIRED_T(bf16_t);
#undef LYP_PAIRED_T
#undef LYP_PAIRED
#undef LYP_PAIRED_KS
  LYP_LAUNCH_CHECK("paired_prefill");
  return 0;
}

// part_keys: from lyp_paired_decode_plan.  With max_parts > 1 part_o needs n_seqs * H * 2 * max_parts * VD floats, part_ml
// n_seqs * H * 2 * max_parts * 2.  Precondition, which only the caller can check (the contexts are on the
// device): no request's token sees more than max_parts * part_keys - 15 keys.
int lyp_paired_decode(const void* q, int q_stride, void* out, int out_stride, const void* kpool, const void* vpool,
                      int dtype, const int32_t* block_tables, int table_width, const int32_t* q_start,
                      const int32_t* ctx_len, const int32_t* dec_seqs, int n_seqs, float* part_o, float* part_ml,
                      int max_parts, int part_keys, int H, int G, int bs, int window, int chunk, float scale, float lambda,
                      float eps, float post, const float* gate, int gate_ld, hipStream_t stream) {
  if (check_common("paired_decode", H, G, bs, table_width, q_stride, out_stride, window, chunk, q, kpool, vpool, gate, gate_ld))
    return -1;
  LYP_REQUIRE(scale > 0.f, "paired_decode: a scale of %g", static_cast<double>(scale));
  LYP_REQUIRE(n_seqs >= 0 && n_seqs <= 65535 && max_parts > 0 && max_parts <= kPartsMost && part_keys > 0 &&
                  part_keys % kDecodeLeast == 0,
              "paired_decode: %d requests, %d partitions of %d keys", n_seqs, max_parts, part_keys);
  LYP_REQUIRE(max_parts == 1 || (part_o && part_ml), "paired_decode: no workspace");
  LYP_REQUIRE(dtype == kF32 || dtype == kBF16, "paired_decode: unknown dtype %d", dtype);
  if (n_seqs == 0) return 0;
  const int g = H / G, col_groups = (g + 15) / 16;
  LYP_REQUIRE(G * col_groups <= 65535, "paired_decode: launch too large");
  const Finish fin{lambda, eps, post, gate, gate_ld};
  const size_t lds = decode_lds_floats(g) * sizeof(float);
  const dim3 grid(max_parts, G * col_groups, n_seqs);
  const float scale_log2 = scale * kLog2e;
#define LYP_PAIRED_DEC_A(T, WHOLE, ALIGNED)                                                                            \
  do {                                                                                                                 \
    if (lds > 48 * 1024) {                                                                                             \
      static bool asked = false;                                                                                       \
      if (!asked) {                                                                                                    \
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(paired_decode_kernel<T, WHOLE, ALIGNED>),              \
                                  hipFuncAttributeMaxDynamicSharedMemorySize,                                          \
                                  static_cast<int>(decode_lds_floats(16) * sizeof(float)));                            \
        asked = true;                                                                                                  \
      }                                                                                                                \
    }                                                                                                                  \
    paired_decode_kernel<T, WHOLE, ALIGNED><<<grid, kDecodeWaves * kWave, lds, stream>>>(                              \
        static_cast<const T*>(q), q_stride, static_cast<const T*>(kpool), static_cast<const T*>(vpool), block_tables,  \
        table_width, q_start, ctx_len, dec_seqs, part_o, part_ml, max_parts, part_keys, H, G, bs, shift_of(bs), window, \
        chunk, scale_log2, static_cast<T*>(out), out_stride, fin);                                                     \
  } while (0)
#define LYP_PAIRED_DEC(T, WHOLE)                             \
  do {                                                       \
    if (bs % 16 == 0) LYP_PAIRED_DEC_A(T, WHOLE, true);      \
    else LYP_PAIRED_DEC_A(T, WHOLE, false);                  \
  } while (0)
#define LYP_PAIRED_DEC_T(T)                                                                                            \
  do {                                                                                                                 \
    if (max_parts == 1) {                                                                                              \
      LYP_PAIRED_DEC(T, true);                                                                                         \
    } else {                                                                                                           \
      LYP_PAIRED_DEC(T, false);                                                                                        \
      paired_merge_decode_kernel<T><<<dim3(H, n_seqs), kMergeThreads, 0, stream>>>(part_o, part_ml, max_parts,         \
                                                                        part_keys, q_start,                            \
                                                                        ctx_len, dec_seqs, static_cast<T*>(out),       \
                                                                        out_stride, H, window, chunk, fin);            \
    }                                                                                                                  \
  } while (0)
  if (dtype == kF32) LYP_PAIRED_DEC_T(float);
  else LYP_PAIRED_DEC_T(bf16_t);
#undef LYP_PAIRED_DEC_T
#undef LYP_PAIRED_DEC
#undef LYP_PAIRED_DEC_A
  LYP_LAUNCH_CHECK("paired_decode");
  return 0;
}

}  // extern "C"
