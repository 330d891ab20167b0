// Attention over a paged cache of latent entries that are kept once: a token's entry is a row of `width` values, the key
// of every head, and the entry's first `kv_rank` values are the value of every head. A page is [P, width].
//
// The general kernel: any element type, any sizes. One block of four waves per (token, head). Keys are walked in tiles of
// 64 that start at multiples of 64, wave w taking tiles w, w + 4, ... of those the query sees; a lane takes one key of a
// tile for its score, then the lanes turn to the value columns (neighbouring lanes read neighbouring values of an entry)
// and weigh them with the tile's weights, handed round from the lanes that hold them. Every wave keeps a running maximum,
// sum and weighted values; the four are combined at the end in wave order, the sink joining there. Which keys a wave takes
// and in which order is decided by the query's position alone. Scores, weights and sums are float32.
#include "common.h"
#include "holon_hip.h"

#define LAT_MAX 1024

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
}  // namespace

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
