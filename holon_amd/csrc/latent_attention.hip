// Attention over a paged cache of latent entries that are kept once: a token's entry is a row of `width` values, the key
// of every head, and the entry's first `kv_rank` values are the value of every head. A page is [P, width].
//
// The general kernel: any element type, any sizes. One block of four waves per (token, head). Keys are walked in tiles of
// 64 that start at multiples of 64, wave w taking tiles w, w + 4, ... of those the query sees; a lane takes one key of a
// tile for its score, then the lanes turn to the value columns (neighbouring lanes read neighbouring values of an entry)
// and weigh them with the tile's weights, handed round from the lanes that hold them. Every wave keeps a running maximum,
// sum and weighted values; the four are combined at the end in wave order, the sink joining there. Which keys a wave takes
// and in which order is decided by the query's position alone. Scores, weights and sums are float32.
//
// The matrix-core kernels (bfloat16, no window): prompt portions and decode rows, below.
#include "common.h"
#include "holon_hip.h"

#define LAT_MAX 1024

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4_t __attribute__((ext_vector_type(4)));
typedef short s16x4_t __attribute__((ext_vector_type(4)));
typedef float f32x4_t __attribute__((ext_vector_type(4)));

namespace {

template <typename T>
__global__ void __launch_bounds__(256) latent_attention_kernel(
    const T* __restrict__ q, T* __restrict__ out, const T* __restrict__ pages, const int32_t* __restrict__ table,
    int table_stride, int table_rows, const int32_t* __restrict__ slots, const int32_t* __restrict__ token_row,
    const int32_t* __restrict__ positions, int heads, int width, int kv_rank, int page_size, int num_pages,
    const float* __restrict__ sink, float scale, int window, int key_vec) {
  __shared__ float q_s[LAT_MAX];
  __shared__ float sum_s[4][LAT_MAX];
  __shared__ float ml_s[4][2];
  const int w = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  const int t = blockIdx.x, h = blockIdx.y;
  const int pos = positions[t];
  int slot = slots[token_row[t]];
  slot = slot < 0 ? 0 : (slot >= table_rows ? table_rows - 1 : slot);
  const int32_t* trow = table + (int64_t)slot * table_stride;
  const T* qp = q + ((int64_t)t * heads + h) * width;
  for (int d = threadIdx.x; d < width; d += 256) q_s[d] = Elem<T>::load(qp[d]);
  __syncthreads();
  const int first = window > 0 ? max(0, pos - window + 1) : 0;
  float m = -INFINITY, l = 0.f;
  float acc[LAT_MAX / WAVE];
#pragma unroll
  for (int i = 0; i < LAT_MAX / WAVE; ++i) acc[i] = 0.f;
  constexpr int VEC = Elem<T>::kVec;
  for (int n = first / WAVE + w; n <= pos / WAVE; n += 4) {
    const int j0 = n * WAVE, key = j0 + lane;
    int64_t entry = -1;
    if (key <= pos && key >= first && key / page_size < table_stride) {
      const int page = trow[key / page_size];
      if (page >= 0 && page < num_pages) entry = ((int64_t)page * page_size + key % page_size) * width;
    }
    float s = -INFINITY;
    if (entry >= 0) {
      const T* kp = pages + entry;
      float dot = 0.f;
      if (key_vec) {
        for (int d = 0; d < width; d += VEC) {
          const uint4 raw = *reinterpret_cast<const uint4*>(kp + d);
          const T* e = reinterpret_cast<const T*>(&raw);
#pragma unroll
          for (int i = 0; i < VEC; ++i) dot += q_s[d + i] * Elem<T>::load(e[i]);
        }
      } else {
        for (int d = 0; d < width; ++d) dot += q_s[d] * Elem<T>::load(kp[d]);
      }
      s = dot * scale;
    }
    const float m_new = fmaxf(m, wave_max(s));
    if (m_new == -INFINITY) continue;                    // nothing seen in this tile (the same in every lane)
    const float alpha = expf(m - m_new);                 // m = -inf before the first key: 0
    const float p = entry >= 0 ? expf(s - m_new) : 0.f;
    l = l * alpha + wave_sum(p);
    m = m_new;
#pragma unroll
    for (int i = 0; i < LAT_MAX / WAVE; ++i) acc[i] *= alpha;
    uint64_t have = __ballot(entry >= 0);                // the lanes whose key is seen and held
    while (have) {
      const int j = __builtin_ctzll(have);
      have &= have - 1;
      const uint32_t lo = __builtin_amdgcn_readlane((uint32_t)entry, j), hi = __builtin_amdgcn_readlane((uint32_t)(entry >> 32), j);
      const float pj = __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(p), j));
      const T* vp = pages + (int64_t)(((uint64_t)hi << 32) | lo);
#pragma unroll
      for (int i = 0; i < LAT_MAX / WAVE; ++i) {
        if (i * WAVE >= kv_rank) break;
        const int d = lane + i * WAVE;
        if (d < kv_rank) acc[i] += pj * Elem<T>::load(vp[d]);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < LAT_MAX / WAVE; ++i) {
    const int d = lane + i * WAVE;
    if (d < kv_rank) sum_s[w][d] = acc[i];
  }
  if (lane == 0) { ml_s[w][0] = m; ml_s[w][1] = l; }
  __syncthreads();
  float top = sink ? sink[h] : -INFINITY;
#pragma unroll
  for (int i = 0; i < 4; ++i) top = fmaxf(top, ml_s[i][0]);
  float f[4], den = 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    f[i] = ml_s[i][0] == -INFINITY ? 0.f : expf(ml_s[i][0] - top);
    den += ml_s[i][1] * f[i];
  }
  if (sink) den += expf(sink[h] - top);
  const float inv = den > 0.f ? 1.0f / den : 0.f;
  for (int d = threadIdx.x; d < kv_rank; d += 256) {
    const float o = ((sum_s[0][d] * f[0] + sum_s[1][d] * f[1]) + sum_s[2][d] * f[2]) + sum_s[3][d] * f[3];
    out[((int64_t)t * heads + h) * kv_rank + d] = Elem<T>::store(o * inv);
  }
}

// -- on the matrix cores ------------------------------------------------------------------------------------------------
// A tile's 16 rows are (token, head) pairs in the order they lie in: all heads read the same entries, so a row is no more
// than a query of `width` values at a position. Operands (v_mfma_f32_16x16x32_bf16: lane l = 16 g + c holds eight values
// of row / column c; the result's lane holds rows 4 g + r, r < 4, of column c):
//   S^T = E Q^T     A = 16 entries x 32 of their values, rows as they lie; two products cover 32 keys, and lane (g, c)
//                   then holds the scores of keys 4 g + r and 16 + 4 g + r of query c. In that order of the inner
//                   dimension they are the B operand of
//   O^T = E_c^T P^T A = 16 of the latent's values x 32 keys: the entries' columns, which ds_read_b64_tr_b16 reads out of
//                   LDS transposed (16 lanes give the addresses of 4 rows x 16 values and get a column's 4 rows each).
// So an entry lies in memory once and in LDS once, and serves both products from there.
// Entries come into LDS by the memory pipeline (16 bytes a lane, a wave's 64 lanes into one contiguous kilobyte). A row's
// pitch in LDS is WP / 2 + 8 words, 8 times an odd number: eight neighbouring rows then start 8 banks apart, which keeps
// the transposed reads and the row reads free of conflicts. A row's columns from `width` on repeat its last ones (the
// query is zero there); rows past the last key repeat the last key's entry (their weights are zero).
// RP, WP: the latent's and the entry's widths, padded to the next sizes that are compiled.
struct LatArgs {
  const bf16_t* q;
  bf16_t* out;
  const bf16_t* pages;
  const int32_t* table;
  const int32_t* slots;
  const int32_t* lens;
  const int32_t* qstart;
  const int32_t* row_ids;
  const float* sink;
  float* part_o;
  float* part_ml;
  int table_stride, table_rows, num_pages, page_size, heads, width, kv_rank;
  int per, splits;             // decode rows: keys a block takes (a multiple of 64), blocks a (row, 16 heads)
  float scale_log2;
};

__device__ __forceinline__ bf16x4_t read_transposed(const unsigned char* p) {
  typedef __attribute__((address_space(3))) s16x4_t* lds_ptr;
  return __builtin_bit_cast(bf16x4_t, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_ptr)p));
}

__device__ __forceinline__ float max_over_groups(float v) {   // over the four lane groups of 16
  const auto rows = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  v = fmaxf(__uint_as_float(rows[0]), __uint_as_float(rows[1]));
  const auto halves = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  return fmaxf(__uint_as_float(halves[0]), __uint_as_float(halves[1]));
}

// KEYS entries on their way into one buffer: what each lane of a block of WAVES waves copies.
template <int WP, int KEYS, int WAVES>
struct EntryCopies {
  static constexpr int PC = WP / 8 + 2;                  // 16-byte pieces a row takes in LDS
  static constexpr int PITCH = PC * 16, BYTES = KEYS * PITCH, NI = KEYS * PC / 64, CI = (NI + WAVES - 1) / WAVES;
  static_assert(KEYS * PC % 64 == 0 && (PC / 2) % 2 == 1, "whole kilobytes, an odd multiple of 8 words a row");
  uint32_t lds0;
  int wave, row0, col0, last;                            // of this lane's first piece; the entry's last piece
  __device__ __forceinline__ void init(const unsigned char* lds, int width) {
    wave = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
    lds0 = (uint32_t)(uintptr_t)(__attribute__((address_space(3))) const void*)lds;
    row0 = threadIdx.x / PC;
    col0 = threadIdx.x % PC;
    last = width / 8 - 1;
  }
  // `from`: the byte offset of every row's entry among the pages, in LDS. (A lane's pieces are WAVES x 64 apart: its next row and
  // column are found as it goes, which costs less than registers held through the kernel.)
  __device__ __forceinline__ void copy(const bf16_t* pages, const int64_t* from, uint32_t buffer) const {
    int row = row0, col = col0;
#pragma unroll
    for (int i = 0; i < CI; ++i) {
      if (wave + WAVES * i >= NI) break;                     // (the same in all of a wave's lanes)
      load_to_lds16_from(reinterpret_cast<const unsigned char*>(pages) + from[row] + min(col, last) * 16,
                         __builtin_amdgcn_readfirstlane(lds0 + buffer + (uint32_t)(wave + WAVES * i) * 1024));
      row += WAVES * 64 / PC;
      col += WAVES * 64 % PC;
      if (col >= PC) { col -= PC; ++row; }
    }
  }
};

// The byte offset of a key's entry (an id the pool does not have reads page 0: nothing outside the pages is touched).
__device__ __forceinline__ int64_t entry_at(const LatArgs& a, int page, int key) {
  page = page < 0 || page >= a.num_pages ? 0 : page;
  return ((int64_t)page * a.page_size + key % a.page_size) * a.width * 2;
}

__device__ __forceinline__ const int32_t* table_row(const LatArgs& a, int b) {
  int slot = a.slots[b];
  slot = slot < 0 ? 0 : (slot >= a.table_rows ? a.table_rows - 1 : slot);
  return a.table + (int64_t)slot * a.table_stride;
}

// Prompt portions: a block of eight waves owns 64 consecutive rows (four tiles) and walks the keys in stages of 32, the
// next stage on its way into one buffer while the other is worked on. Wave w scores tile w / 2 against half w % 2 of the
// stage's keys; maxima and weights meet in LDS; then wave w sums a quarter of the latent's columns (w / 2) for two tiles
// (w % 2): a transposed read serves two tiles, and a wave's sums take the registers of half a tile, which leaves room for
// a stage's operands to be asked for ahead of the products. Long rows come first.
template <int RP, int WP>
__global__ void __launch_bounds__(512, 2) latent_prefill_kernel(LatArgs a) {
  using EC = EntryCopies<WP, 32, 8>;
  constexpr int KS = WP / 32, DQ = RP / 64, PG = 1024;   // DQ: d-tiles of 16 a wave
  __shared__ __attribute__((aligned(1024))) unsigned char stage_lds[2 * EC::BYTES];
  __shared__ int64_t from_s[2][32];
  __shared__ int32_t pg_s[PG];
  __shared__ float max_s[2][64], alpha_s[64];
  __shared__ __attribute__((aligned(16))) bf16_t p_s[4][2][4][16][4];  // [tile][half of the keys][lane group][row][key]
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid % WAVE, g = lane / 16, c = lane % 16;
  const int rt = wave / 2, kh = wave % 2;
  const int b = a.row_ids[blockIdx.y];
  const int qs = a.qstart[b], nq = a.qstart[b + 1] - qs, n = a.lens[b];
  const int rows = nq * a.heads, tiles = (rows + 63) / 64;
  if ((int)blockIdx.x >= tiles || n <= 0) return;        // (the same in all of the block's threads)
  const int range = tiles - 1 - blockIdx.x;
  const int32_t* trow = table_row(a, b);
  for (int i = tid; i < min(PG, a.table_stride); i += 512) pg_s[i] = trow[i];
  const int m0 = range * 64, row = m0 + rt * 16 + c, before = n - nq;
  const bool valid = row < rows;
  const int ti = valid ? row / a.heads : 0, head = valid ? row % a.heads : 0;
  const int qpos = valid ? before + ti : -1;
  const int blk_first = before + m0 / a.heads;
  const int key_hi = before + (min(rows, m0 + 64) - 1) / a.heads, kb_last = key_hi / 32 * 32;
  EC ec;
  ec.init(stage_lds, a.width);
  bf16x8_t qf[KS];
  {
    const bf16_t* qp = a.q + ((int64_t)(qs + ti) * a.heads + head) * a.width + 8 * g;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      if (valid && ks * 32 + 8 * g < a.width) qf[ks] = *reinterpret_cast<const bf16x8_t*>(qp + ks * 32);
      else
#pragma unroll
        for (int i = 0; i < 8; ++i) qf[ks][i] = (__bf16)0.f;
    }
  }
  f32x4_t o[DQ][2];
#pragma unroll
  for (int d = 0; d < DQ; ++d) o[d][0] = o[d][1] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;                          // of this wave's row c: the maximum over all keys, its half's sum
  lds_barrier();                                         // the block's table is in LDS
  auto find = [&](int kb, int buf) {                     // where the entries of the stage at kb lie
    if (tid < 32) {
      const int key = min(kb + tid, n - 1), at = min(key / a.page_size, a.table_stride - 1);
      int page;
      if (at < PG) page = pg_s[at];
      else page = trow[at];
      from_s[buf][tid] = entry_at(a, page, key);
    }
  };
  find(0, 0);
  find(32, 1);
  lds_barrier();
  ec.copy(a.pages, from_s[0], 0);
  wait_loads_but<0>();
  lds_barrier();
  for (int kb = 0, buf = 0; kb <= kb_last; kb += 32, buf ^= 1) {
    if (kb < kb_last) ec.copy(a.pages, from_s[buf ^ 1], (uint32_t)(buf ^ 1) * EC::BYTES);
    if (kb + 32 < kb_last) find(kb + 64, buf);           // (this stage's own places have been read a stage ago)
    const unsigned char* lds = stage_lds + buf * EC::BYTES;
    float sv[4];
    {
      const unsigned char* kp = lds + (16 * kh + c) * EC::PITCH + g * 16;
      f32x4_t s0 = f32x4_t{0.f, 0.f, 0.f, 0.f}, s1 = s0;
      bf16x8_t kf[KS];
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) kf[ks] = *reinterpret_cast<const bf16x8_t*>(kp + ks * 64);
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        f32x4_t& s = ks % 2 ? s1 : s0;
        s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[ks], qf[ks], s, 0, 0, 0);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) sv[r] = s0[r] + s1[r];
    }
    if (kb + 31 > blk_first) {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (kb + 16 * kh + 4 * g + r > qpos) sv[r] = -INFINITY;
    }
    const float mx = max_over_groups(fmaxf(fmaxf(sv[0], sv[1]), fmaxf(sv[2], sv[3])));
    if (g == 0) max_s[kh][rt * 16 + c] = mx * a.scale_log2;
    lds_barrier();
    {
      const float m_new = fmaxf(m, fmaxf(max_s[0][rt * 16 + c], max_s[1][rt * 16 + c]));
      const float m_use = m_new == -INFINITY ? 0.f : m_new;
      const float alpha = __builtin_amdgcn_exp2f(m - m_use);
      float p[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) p[r] = __builtin_amdgcn_exp2f(fmaf(sv[r], a.scale_log2, -m_use));
      ushort4 w;
      w.x = float_to_bf16(p[0]); w.y = float_to_bf16(p[1]); w.z = float_to_bf16(p[2]); w.w = float_to_bf16(p[3]);
      *reinterpret_cast<ushort4*>(&p_s[rt][kh][g][c][0]) = w;
      if (kh == 0 && g == 0) alpha_s[rt * 16 + c] = alpha;
      l = l * alpha + ((p[0] + p[1]) + (p[2] + p[3]));
      m = m_new;
    }
    lds_barrier();
    {
      bf16x8_t pb[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) {                      // tiles 2 kh and 2 kh + 1
        const bf16x4_t lo = *reinterpret_cast<const bf16x4_t*>(&p_s[2 * kh + i][0][g][c][0]);
        const bf16x4_t hi = *reinterpret_cast<const bf16x4_t*>(&p_s[2 * kh + i][1][g][c][0]);
        pb[i] = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
        const float alpha = alpha_s[(2 * kh + i) * 16 + c];
        if (__any(alpha != 1.f)) {
#pragma unroll
          for (int d = 0; d < DQ; ++d) o[d][i] *= alpha;
        }
      }
      const unsigned char* vp = lds + (4 * g + c / 4) * EC::PITCH + (c % 4) * 8 + rt * DQ * 32;
      bf16x8_t v[DQ];
#pragma unroll
      for (int d = 0; d < DQ; ++d)
        v[d] = __builtin_shufflevector(read_transposed(vp + d * 32), read_transposed(vp + 16 * EC::PITCH + d * 32), 0, 1, 2, 3, 4,
                                       5, 6, 7);
#pragma unroll
      for (int d = 0; d < DQ; ++d) {
        o[d][0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v[d], pb[0], o[d][0], 0, 0, 0);
        o[d][1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v[d], pb[1], o[d][1], 0, 0, 0);
      }
    }
    wait_loads_but<0>();                                 // the next stage has landed (this wave's share of it)
    lds_barrier();
  }
  l += __shfl_xor(l, 16, WAVE);
  l += __shfl_xor(l, 32, WAVE);
  if (g == 0) max_s[kh][rt * 16 + c] = l;
  if (g == 0 && kh == 0) alpha_s[rt * 16 + c] = valid && a.sink ? __builtin_amdgcn_exp2f(a.sink[head] * 1.4426950408889634f - m) : 0.f;
  lds_barrier();
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int at = (2 * kh + i) * 16 + c, r = m0 + at;
    if (r >= rows) continue;
    const float den = (max_s[0][at] + max_s[1][at]) + alpha_s[at];
    const float inv = den > 0.f ? 1.0f / den : 0.f;
    const int d0 = rt * DQ * 16 + 4 * g;
    bf16_t* op = a.out + ((int64_t)qs * a.heads + r) * a.kv_rank + d0;
#pragma unroll
    for (int d = 0; d < DQ; ++d) {
      if (d0 + d * 16 >= a.kv_rank) break;
      ushort4 w;
      w.x = float_to_bf16(o[d][i][0] * inv);
      w.y = float_to_bf16(o[d][i][1] * inv);
      w.z = float_to_bf16(o[d][i][2] * inv);
      w.w = float_to_bf16(o[d][i][3] * inv);
      *reinterpret_cast<ushort4*>(op + d * 16) = w;
    }
  }
}

// Decode rows: a block of four waves takes a share of a row's keys for 16 heads, 64 keys at a time: wave w scores keys
// 16 w .. 16 w + 15, the maxima and the weights meet in LDS, and wave w sums a quarter of the latent's columns over all 64.
// One block a row writes the result; more leave (values, maximum, sum) for the merge below.
template <int RP, int WP>
__global__ void __launch_bounds__(256, 2) latent_decode_kernel(LatArgs a) {
  using EC = EntryCopies<WP, 64, 4>;
  constexpr int KS = WP / 32, DW = RP / 64;              // d-tiles of 16 a wave
  __shared__ __attribute__((aligned(1024))) unsigned char tile_lds[EC::BYTES];
  __shared__ int64_t from_s[64];
  __shared__ float red_s[4][16];
  __shared__ __attribute__((aligned(8))) bf16_t p_s[4][4][16][4];      // [wave][lane group][head][key of the four]
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid % WAVE, g = lane / 16, c = lane % 16;
  const int b = a.row_ids[blockIdx.z], split = blockIdx.x, h0 = blockIdx.y * 16;
  const int n = a.lens[b], token = a.qstart[b];
  const int lo = split * a.per, hi = min(n, lo + a.per);             // keys lo .. hi - 1
  const int head = h0 + c;
  const bool valid = head < a.heads;
  const int64_t cell = ((int64_t)blockIdx.z * a.heads + (valid ? head : 0)) * a.splits + split;
  if (lo >= hi) {                                        // (the same in all of the block's threads) nothing of this row
    if (a.splits > 1 && tid < 16 && valid) { a.part_ml[cell * 2] = -INFINITY; a.part_ml[cell * 2 + 1] = 0.f; }
    return;
  }
  const int32_t* trow = table_row(a, b);
  EC ec;
  ec.init(tile_lds, a.width);
  bf16x8_t qf[KS];
  {
    const bf16_t* qp = a.q + ((int64_t)token * a.heads + (valid ? head : 0)) * a.width + 8 * g;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      if (valid && ks * 32 + 8 * g < a.width) qf[ks] = *reinterpret_cast<const bf16x8_t*>(qp + ks * 32);
      else
#pragma unroll
        for (int i = 0; i < 8; ++i) qf[ks][i] = (__bf16)0.f;
    }
  }
  f32x4_t o[DW];
#pragma unroll
  for (int d = 0; d < DW; ++d) o[d] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  for (int kb = lo; kb < hi; kb += 64) {
    if (tid < 64) {
      const int key = min(kb + tid, hi - 1);
      from_s[tid] = entry_at(a, trow[min(key / a.page_size, a.table_stride - 1)], key);
    }
    lds_barrier();                                       // (and every wave has left the tile before)
    ec.copy(a.pages, from_s, 0);
    wait_loads_but<0>();
    lds_barrier();
    const unsigned char* kp = tile_lds + (16 * wave + c) * EC::PITCH + g * 16;
    f32x4_t s0 = f32x4_t{0.f, 0.f, 0.f, 0.f}, s1 = s0;
#pragma unroll
    for (int ks = 0; ks < KS; ks += 2) {
      s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8_t*>(kp + ks * 64), qf[ks], s0, 0, 0, 0);
      if (ks + 1 < KS)
        s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8_t*>(kp + ks * 64 + 64),
                                                     qf[ks + 1 < KS ? ks + 1 : 0], s1, 0, 0, 0);
    }
    float sv[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) sv[r] = kb + 16 * wave + 4 * g + r < hi ? s0[r] + s1[r] : -INFINITY;
    const float mx = max_over_groups(fmaxf(fmaxf(sv[0], sv[1]), fmaxf(sv[2], sv[3])));
    if (g == 0) red_s[wave][c] = mx * a.scale_log2;
    lds_barrier();
    const float m_new = fmaxf(fmaxf(fmaxf(red_s[0][c], red_s[1][c]), fmaxf(red_s[2][c], red_s[3][c])), m);
    const float alpha = __builtin_amdgcn_exp2f(m - m_new);           // (a tile holds at least one key: m_new is finite)
    m = m_new;
    l *= alpha;
    ushort4 w;
    float p[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) { p[r] = __builtin_amdgcn_exp2f(fmaf(sv[r], a.scale_log2, -m)); l += p[r]; }
    w.x = float_to_bf16(p[0]); w.y = float_to_bf16(p[1]); w.z = float_to_bf16(p[2]); w.w = float_to_bf16(p[3]);
    *reinterpret_cast<ushort4*>(&p_s[wave][g][c][0]) = w;
#pragma unroll
    for (int d = 0; d < DW; ++d) o[d] *= alpha;
    lds_barrier();
#pragma unroll
    for (int j = 0; j < 2; ++j) {                        // 32 keys: those of waves 2 j and 2 j + 1
      const bf16x4_t plo = *reinterpret_cast<const bf16x4_t*>(&p_s[2 * j][g][c][0]);
      const bf16x4_t phi = *reinterpret_cast<const bf16x4_t*>(&p_s[2 * j + 1][g][c][0]);
      const bf16x8_t pb = __builtin_shufflevector(plo, phi, 0, 1, 2, 3, 4, 5, 6, 7);
      const unsigned char* vp = tile_lds + (32 * j + 4 * g + c / 4) * EC::PITCH + (c % 4) * 8 + wave * DW * 32;
#pragma unroll
      for (int d = 0; d < DW; ++d) {
        const bf16x4_t vlo = read_transposed(vp + d * 32), vhi = read_transposed(vp + 16 * EC::PITCH + d * 32);
        o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_shufflevector(vlo, vhi, 0, 1, 2, 3, 4, 5, 6, 7), pb, o[d],
                                                       0, 0, 0);
      }
    }
  }
  l += __shfl_xor(l, 16, WAVE);
  l += __shfl_xor(l, 32, WAVE);
  lds_barrier();                                         // every wave has read the last maxima
  if (g == 0) red_s[wave][c] = l;
  lds_barrier();
  l = (red_s[0][c] + red_s[1][c]) + (red_s[2][c] + red_s[3][c]);
  if (!valid) return;
  const int d0 = wave * DW * 16 + 4 * g;
  if (a.splits > 1) {
    if (wave == 0 && g == 0) { a.part_ml[cell * 2] = m; a.part_ml[cell * 2 + 1] = l; }
    float* op = a.part_o + cell * a.kv_rank + d0;
#pragma unroll
    for (int d = 0; d < DW; ++d)
      if (d0 + d * 16 < a.kv_rank) *reinterpret_cast<f32x4_t*>(op + d * 16) = o[d];
    return;
  }
  if (a.sink) l += __builtin_amdgcn_exp2f(a.sink[head] * 1.4426950408889634f - m);
  const float inv = l > 0.f ? 1.0f / l : 0.f;
  bf16_t* op = a.out + ((int64_t)token * a.heads + head) * a.kv_rank + d0;
#pragma unroll
  for (int d = 0; d < DW; ++d) {
    if (d0 + d * 16 >= a.kv_rank) break;
    ushort4 w;
    w.x = float_to_bf16(o[d][0] * inv);
    w.y = float_to_bf16(o[d][1] * inv);
    w.z = float_to_bf16(o[d][2] * inv);
    w.w = float_to_bf16(o[d][3] * inv);
    *reinterpret_cast<ushort4*>(op + d * 16) = w;
  }
}

// out = sum_i 2^(m_i - M) o_i / sum_i 2^(m_i - M) l_i over a (decode row, head)'s splits (at most 64), the sink joining the
// denominator. A block a (row, head, 128 columns): thread (side, column) takes four columns of splits side, side + 8, ...,
// all asked for before the factors are known; the eight sides are added in order.
__global__ void __launch_bounds__(256) latent_merge_kernel(LatArgs a) {
  constexpr int SIDES = 8, EACH = 64 / SIDES;
  __shared__ float f_s[64];
  __shared__ float den_s;
  __shared__ __attribute__((aligned(16))) f32x4_t sum_s[SIDES][32];
  const int head = blockIdx.x, tid = threadIdx.x, b = a.row_ids[blockIdx.y];
  const int64_t cell = ((int64_t)blockIdx.y * a.heads + head) * a.splits;
  const int side = tid / 32, d = blockIdx.z * 128 + (tid % 32) * 4;
  const bool held = d < a.kv_rank;
  f32x4_t v[EACH];
#pragma unroll
  for (int e = 0; e < EACH; ++e)
    if (held && side + SIDES * e < a.splits)
      v[e] = *reinterpret_cast<const f32x4_t*>(a.part_o + (cell + side + SIDES * e) * a.kv_rank + d);
  if (tid < WAVE) {
    const float mi = tid < a.splits ? a.part_ml[(cell + tid) * 2] : -INFINITY;
    const float li = tid < a.splits ? a.part_ml[(cell + tid) * 2 + 1] : 0.f;
    const float top = wave_max(mi);
    const float f = mi == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(mi - top);
    f_s[tid] = f;
    float den = wave_sum(f * li);
    if (a.sink) den += __builtin_amdgcn_exp2f(a.sink[head] * 1.4426950408889634f - top);
    if (tid == 0) den_s = den > 0.f ? 1.0f / den : 0.f;
  }
  __syncthreads();
  f32x4_t acc = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int e = 0; e < EACH; ++e) {
    if (!held || side + SIDES * e >= a.splits) break;
    const float f = f_s[side + SIDES * e];               // (a split that saw nothing has written no values: not used)
    if (f != 0.f) acc += f * v[e];
  }
  sum_s[side][tid % 32] = acc;
  __syncthreads();
  if (side > 0 || !held) return;
#pragma unroll
  for (int i = 1; i < SIDES; ++i) acc += sum_s[i][tid];
  const float inv = den_s;
  ushort4 w;
  w.x = float_to_bf16(acc[0] * inv); w.y = float_to_bf16(acc[1] * inv);
  w.z = float_to_bf16(acc[2] * inv); w.w = float_to_bf16(acc[3] * inv);
  *reinterpret_cast<ushort4*>(a.out + ((int64_t)a.qstart[b] * a.heads + head) * a.kv_rank + d) = w;
}

// -- every head's own projection ------------------------------------------------------------------------------------------
// y[t, h, b] = sum_a x[t, h, a] w[h, b, a], bfloat16 operands, float32 sums, one rounding; with `gate` the sum times
// sigmoid(gate[t, h B + b]) first. A = 16 rows of w x 32, B = 32 x 16 tokens: a lane holds four neighbouring results of a
// token. Rows past B or the last token repeat the last one that is there; their results are not stored.
struct HeadLinear {
  const bf16_t* x;
  const bf16_t* w;
  bf16_t* y;
  const bf16_t* gate;
  int64_t gate_stride;
  int rows, heads, A, B, y_head;
  int wide_out, wide_gate;     // four results (few tokens) or eight (many) lie on a border of their size, gates likewise
};

// Eight values from column k + 8 g of a row on (`row` points at column 8 g). TAIL: A is no multiple of 32, and a piece past
// the row's end counts as zeros (it is read from the row's start all the same: a branch around a load would keep the loads
// from being under way together).
template <bool TAIL>
__device__ __forceinline__ bf16x8_t load_piece(const bf16_t* row, int k, int g, int A) {
  if constexpr (!TAIL) return *reinterpret_cast<const bf16x8_t*>(row + k);
  const bool ok = k + 8 * g < A;
  uint4 v = *reinterpret_cast<const uint4*>(row + (ok ? k : -8 * g));
  v.x = ok ? v.x : 0u; v.y = ok ? v.y : 0u; v.z = ok ? v.z : 0u; v.w = ok ? v.w : 0u;
  return __builtin_bit_cast(bf16x8_t, v);
}

__device__ __forceinline__ void head_linear_store(const HeadLinear& a, int t, int h, int b, f32x4_t v) {
  if (t >= a.rows || b >= a.B) return;
  if (a.gate) {
    const bf16_t* gp = a.gate + t * a.gate_stride + (int64_t)h * a.B + b;
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (b + r < a.B) v[r] *= __builtin_amdgcn_rcpf(1.0f + __expf(-bf16_to_float(gp[r])));
  }
  bf16_t* yp = a.y + ((int64_t)t * a.heads + h) * a.y_head + b;
  if (a.wide_out && b + 3 < a.B) {
    ushort4 o;
    o.x = float_to_bf16(v[0]); o.y = float_to_bf16(v[1]); o.z = float_to_bf16(v[2]); o.w = float_to_bf16(v[3]);
    *reinterpret_cast<ushort4*>(yp) = o;
  } else {
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (b + r < a.B) yp[r] = float_to_bf16(v[r]);
  }
}

// Up to 16 tokens: a block a head and 16 columns, A dealt to its four waves in steps of 32, their sums added in wave order.
template <bool TAIL>
__global__ void __launch_bounds__(256) head_linear_few_kernel(HeadLinear a) {
  __shared__ f32x4_t sum_s[3][WAVE];
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE, g = lane / 16, c = lane % 16;
  const int h = blockIdx.x, b0 = blockIdx.y * 16;
  const bf16_t* wp = a.w + ((int64_t)h * a.B + min(b0 + c, a.B - 1)) * a.A + 8 * g;
  const bf16_t* xp = a.x + ((int64_t)min(c, a.rows - 1) * a.heads + h) * a.A + 8 * g;
  f32x4_t acc = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int k = wave * 32; k < a.A; k += 128) {
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(load_piece<TAIL>(wp, k, g, a.A), load_piece<TAIL>(xp, k, g, a.A), acc, 0, 0, 0);
  }
  if (wave > 0) sum_s[wave - 1][lane] = acc;
  __syncthreads();
  if (wave > 0) return;
  acc = ((acc + sum_s[0][lane]) + sum_s[1][lane]) + sum_s[2][lane];
  head_linear_store(a, c, h, b0 + 4 * g, acc);
}

// More tokens: a block 128 tokens and 128 columns of a head, a wave 64 by 64; a step's operands are asked for while the
// step before is multiplied. The results pass LDS on their way out, half of a wave's tokens at a time, so that a token's 64
// columns are stored as one whole line and its gates are read as one.
template <bool TAIL>
__global__ void __launch_bounds__(256) head_linear_many_kernel(HeadLinear a) {
  constexpr int OP = 68;
  __shared__ __attribute__((aligned(16))) float out_s[4][32 * OP];
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE, g = lane / 16, c = lane % 16;
  const int h = blockIdx.y, t0 = blockIdx.x * 128 + (wave % 2) * 64, b0 = blockIdx.z * 128 + (wave / 2) * 64;
  if (b0 >= a.B || t0 >= a.rows) return;
  const bf16_t* wp[4];
  const bf16_t* xp[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    wp[i] = a.w + ((int64_t)h * a.B + min(b0 + 16 * i + c, a.B - 1)) * a.A + 8 * g;
    xp[i] = a.x + ((int64_t)min(t0 + 16 * i + c, a.rows - 1) * a.heads + h) * a.A + 8 * g;
  }
  f32x4_t acc[4][4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  bf16x8_t wf[2][4], xf[2][4];
  auto ask = [&](int k, int buf) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      wf[buf][i] = load_piece<TAIL>(wp[i], k, g, a.A);
      xf[buf][i] = load_piece<TAIL>(xp[i], k, g, a.A);
    }
  };
  auto multiply = [&](int buf) {
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j)
        acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[buf][i], xf[buf][j], acc[i][j], 0, 0, 0);
  };
  ask(0, 0);
  for (int k = 0; k < a.A; k += 64) {
    if (k + 32 < a.A) ask(k + 32, 1);
    multiply(0);
    if (k + 64 < a.A) ask(k + 64, 0);
    if (k + 32 < a.A) multiply(1);
  }
  float* mine = out_s[wave];                             // (a wave's own: its LDS operations run in order)
  const int piece = (lane % 8) * 8, b = b0 + piece;
#pragma unroll
  for (int part = 0; part < 2; ++part) {
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int i = 0; i < 4; ++i) *reinterpret_cast<f32x4_t*>(mine + (16 * j + c) * OP + 16 * i + 4 * g) = acc[i][2 * part + j];
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int at = e * 8 + lane / 8, t = t0 + part * 32 + at;
      if (t >= a.rows || b >= a.B) continue;
      float v[8];
      *reinterpret_cast<f32x4_t*>(v) = *reinterpret_cast<const f32x4_t*>(mine + at * OP + piece);
      *reinterpret_cast<f32x4_t*>(v + 4) = *reinterpret_cast<const f32x4_t*>(mine + at * OP + piece + 4);
      const bool whole = b + 7 < a.B;
      if (a.gate) {
        const bf16_t* gp = a.gate + t * a.gate_stride + (int64_t)h * a.B + b;
        __attribute__((aligned(16))) bf16_t gv[8];
        if (whole && a.wide_gate) *reinterpret_cast<uint4*>(gv) = *reinterpret_cast<const uint4*>(gp);
        else
#pragma unroll
          for (int u = 0; u < 8; ++u) gv[u] = b + u < a.B ? gp[u] : (bf16_t)0;
#pragma unroll
        for (int u = 0; u < 8; ++u) v[u] *= __builtin_amdgcn_rcpf(1.0f + __expf(-bf16_to_float(gv[u])));
      }
      bf16_t* yp = a.y + ((int64_t)t * a.heads + h) * a.y_head + b;
      if (whole && a.wide_out) {
        uint4 raw;
        bf16_t* o = reinterpret_cast<bf16_t*>(&raw);
#pragma unroll
        for (int u = 0; u < 8; ++u) o[u] = float_to_bf16(v[u]);
        *reinterpret_cast<uint4*>(yp) = raw;
      } else {
#pragma unroll
        for (int u = 0; u < 8; ++u)
          if (b + u < a.B) yp[u] = float_to_bf16(v[u]);
      }
    }
    __builtin_amdgcn_wave_barrier();
  }
}
}  // namespace

// The per-head projection of bfloat16 rows, any number of them (A a multiple of 8, operands on 16-byte borders).
extern "C" int holon_head_linear_bf16(const void* x, const void* w, void* y, int rows, int heads, int A, int B, int y_head,
                                      const void* gate, int64_t gate_stride, void* stream) {
  HOLON_CHECK(rows >= 1 && heads > 0 && heads <= 65535 && A > 0 && A % 8 == 0 && B > 0 && B <= 65535 * 16 && y_head >= B &&
                  (uintptr_t)x % 16 == 0 && (uintptr_t)w % 16 == 0,
              "head_linear: %d rows, %d heads of %d (a multiple of 8) -> %d (in steps of %d)", rows, heads, A, B, y_head);
  const int unit = rows <= 16 ? 4 : 8;                   // results a lane stores at once
  const HeadLinear a{(const bf16_t*)x, (const bf16_t*)w, (bf16_t*)y, (const bf16_t*)gate, gate_stride, rows, heads, A, B, y_head,
                     (int)(y_head % unit == 0 && (uintptr_t)y % (2 * unit) == 0),
                     (int)(gate_stride % 8 == 0 && B % 8 == 0 && (uintptr_t)gate % 16 == 0)};
  hipStream_t s = (hipStream_t)stream;
  const dim3 few(heads, (B + 15) / 16), many((rows + 127) / 128, heads, (B + 127) / 128);
  if (rows <= 16) {
    if (A % 32) head_linear_few_kernel<true><<<few, 256, 0, s>>>(a); else head_linear_few_kernel<false><<<few, 256, 0, s>>>(a);
  } else {
    if (A % 32) head_linear_many_kernel<true><<<many, 256, 0, s>>>(a); else head_linear_many_kernel<false><<<many, 256, 0, s>>>(a);
  }
  HOLON_LAUNCH_OK();
  return 0;
}

#define LAT_BY_SIZE(CALL)                                                                            \
  do {                                                                                               \
    if (kv_rank <= 64 && width <= 96) { constexpr int RP = 64, WP = 96; CALL; }                      \
    else if (kv_rank <= 128 && width <= 160) { constexpr int RP = 128, WP = 160; CALL; }             \
    else if (kv_rank <= 192 && width <= 256) { constexpr int RP = 192, WP = 256; CALL; }             \
    else if (kv_rank <= 256 && width <= 320) { constexpr int RP = 256, WP = 320; CALL; }             \
    else { constexpr int RP = 512, WP = 576; CALL; }                                                 \
  } while (0)

// Whether the matrix-core kernels serve bfloat16 entries of these sizes.
extern "C" int holon_latent_cores_supported(int width, int kv_rank) {
  return kv_rank > 0 && kv_rank % 4 == 0 && kv_rank <= 512 && width % 8 == 0 && width >= kv_rank && width <= 576;
}

static int latent_cores_check(const char* what, int rows, int heads, int width, int kv_rank, int page_size, int num_pages,
                              int table_stride, int table_rows, float scale) {
  HOLON_CHECK(holon_latent_cores_supported(width, kv_rank), "%s: entries of %d (multiples of 8 up to 576) with latents of %d "
              "(multiples of 4 up to 512)", what, width, kv_rank);
  HOLON_CHECK(rows >= 0 && rows <= 65535 && heads > 0 && page_size > 0 && num_pages > 0 && table_stride > 0 && table_rows > 0 &&
                  scale > 0.f, "%s: %d rows of %d heads, pages of %d, scale %g", what, rows, heads, page_size, scale);
  return 0;
}

extern "C" int holon_latent_prefill_bf16(const void* q, void* out, const void* pages, const int32_t* table,
                                         int table_stride, int table_rows, const int32_t* slots, const int32_t* lens,
                                         const int32_t* qstart, const int32_t* row_ids, int rows, int max_query, int heads,
                                         int width, int kv_rank, int page_size, int num_pages, const float* sink,
                                         float scale, void* stream) {
  if (latent_cores_check("latent_prefill", rows, heads, width, kv_rank, page_size, num_pages, table_stride, table_rows, scale))
    return -1;
  HOLON_CHECK(max_query > 0 && (int64_t)max_query * heads <= 0x7fffffff - 64, "latent_prefill: %d tokens of %d heads", max_query,
              heads);
  if (rows == 0) return 0;
  LatArgs a{(const bf16_t*)q, (bf16_t*)out, (const bf16_t*)pages, table, slots, lens, qstart, row_ids, sink, nullptr, nullptr,
            table_stride, table_rows, num_pages, page_size, heads, width, kv_rank, 0, 1, scale * 1.4426950408889634f};
  const dim3 grid((max_query * heads + 63) / 64, rows);
  LAT_BY_SIZE((latent_prefill_kernel<RP, WP><<<grid, 512, 0, (hipStream_t)stream>>>(a)));
  HOLON_LAUNCH_OK();
  return 0;
}

extern "C" int holon_latent_decode_bf16(const void* q, void* out, const void* pages, const int32_t* table,
                                        int table_stride, int table_rows, const int32_t* slots, const int32_t* lens,
                                        const int32_t* qstart, const int32_t* row_ids, int rows, int max_len, int heads,
                                        int width, int kv_rank, int page_size, int num_pages, const float* sink,
                                        float scale, int splits, int per, float* part_o, float* part_ml, void* stream) {
  if (latent_cores_check("latent_decode", rows, heads, width, kv_rank, page_size, num_pages, table_stride, table_rows, scale))
    return -1;
  HOLON_CHECK(splits >= 1 && splits <= 64 && per > 0 && per % 64 == 0 && (int64_t)splits * per >= max_len &&
                  (splits == 1 || (part_o && part_ml)),
              "latent_decode: %d shares of %d keys for rows of up to %d", splits, per, max_len);
  if (rows == 0) return 0;
  LatArgs a{(const bf16_t*)q, (bf16_t*)out, (const bf16_t*)pages, table, slots, lens, qstart, row_ids, sink, part_o, part_ml,
            table_stride, table_rows, num_pages, page_size, heads, width, kv_rank, per, splits, scale * 1.4426950408889634f};
  const dim3 grid(splits, (heads + 15) / 16, rows);
  LAT_BY_SIZE((latent_decode_kernel<RP, WP><<<grid, 256, 0, (hipStream_t)stream>>>(a)));
  HOLON_LAUNCH_OK();
  if (splits > 1) {
    latent_merge_kernel<<<dim3(heads, rows, (kv_rank + 127) / 128), 256, 0, (hipStream_t)stream>>>(a);
    HOLON_LAUNCH_OK();
  }
  return 0;
}

extern "C" int holon_latent_attention(const void* q, void* out, const void* pages, const int32_t* table,
                                      int table_stride, int table_rows, const int32_t* slots, const int32_t* token_row,
                                      const int32_t* positions, int tokens, int heads, int width, int kv_rank,
                                      int page_size, int num_pages, const float* sink, float scale, int window,
                                      int dtype, void* stream) {
  HOLON_CHECK(tokens >= 0 && heads > 0 && heads <= 65535, "latent_attention: %d tokens of %d heads", tokens, heads);
  HOLON_CHECK(kv_rank > 0 && kv_rank <= width && width <= LAT_MAX, "latent_attention: entries of %d (at most %d), latents "
              "of %d", width, LAT_MAX, kv_rank);
  HOLON_CHECK(page_size > 0 && num_pages > 0 && window >= 0 && table_stride > 0 && table_rows > 0,
              "latent_attention: bad page geometry");
  if (tokens == 0) return 0;
  const dim3 grid(tokens, heads);
  hipStream_t s = (hipStream_t)stream;
  const int key_vec = (uintptr_t)pages % 16 == 0 && width % (dtype == HOLON_F32 ? 4 : 8) == 0;
#define LAT_LAUNCH(T)                                                                                                 \
  latent_attention_kernel<T><<<grid, 256, 0, s>>>((const T*)q, (T*)out, (const T*)pages, table, table_stride, table_rows, \
                                                  slots, token_row, positions, heads, width, kv_rank, page_size,     \
                                                  num_pages, sink, scale, window, key_vec)
  if (dtype == HOLON_F32) LAT_LAUNCH(float); else LAT_LAUNCH(bf16_t);
#undef LAT_LAUNCH
  HOLON_LAUNCH_OK();
  return 0;
}
