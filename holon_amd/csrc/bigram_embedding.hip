// An embedding that adds to a token's row the row of a second table chosen by the token and the one before it:
// x = E[t] + B[(prev mul_prev + t mul_cur) mod buckets], a sequence's first token taking row `buckets` (the last one).
// The rows come out in float32. The token before a row's first lies in the request's slot (`prev`), which afterwards
// holds the row's last token; a row that starts at position 0 has none whatever the slot holds.
#include "common.h"
#include "holon_hip.h"

namespace {

__device__ __forceinline__ int token_at(const int32_t* __restrict__ ids, const int32_t* __restrict__ take_slot,
                                        const int32_t* __restrict__ last_token, int t, int vocab) {
  int id = ids[t];
  if (take_slot != nullptr && take_slot[t] >= 0) id = last_token[take_slot[t]];    // drawn by the step before
  return min(max(id, 0), vocab - 1);
}

// One block a token. `keep`: every row has one token and token t is row t; the block then leaves its token in the slot
// (no other block reads that slot).
template <typename T>
__global__ void __launch_bounds__(256) bigram_embedding_kernel(
    const int32_t* __restrict__ ids, const int32_t* __restrict__ take_slot, const int32_t* __restrict__ last_token,
    const T* __restrict__ table, const T* __restrict__ bigram, int32_t* __restrict__ prev,
    const int32_t* __restrict__ slots, const int32_t* __restrict__ starts, const int32_t* __restrict__ query_start,
    const int32_t* __restrict__ token_row, float* __restrict__ y, int width, int vocab, int buckets, int64_t mul_prev,
    int64_t mul_cur, int keep) {
  const int t = blockIdx.x;
  const int b = keep ? t : token_row[t];
  const int q0 = keep ? t : query_start[b];
  const int tok = token_at(ids, take_slot, last_token, t, vocab);
  int before = -1;
  if (t > q0) before = token_at(ids, take_slot, last_token, t - 1, vocab);
  else if (starts[b] > 0) before = prev[slots[b]];
  int64_t row = buckets;
  if (before >= 0) {
    row = ((int64_t)before * mul_prev + (int64_t)tok * mul_cur) % buckets;
    if (row < 0) row += buckets;
  }
  const T* e = table + (int64_t)tok * width;
  const T* g = bigram + row * width;
  float* o = y + (int64_t)t * width;
  constexpr int V = Elem<T>::kVec;
  if (width % V == 0) {                                  // (both tables and y are tensors' starts: 16 bytes)
    for (int i = threadIdx.x * V; i < width; i += 256 * V) {
      const uint4 eraw = *reinterpret_cast<const uint4*>(e + i), graw = *reinterpret_cast<const uint4*>(g + i);
      const T* ev = reinterpret_cast<const T*>(&eraw);
      const T* gv = reinterpret_cast<const T*>(&graw);
#pragma unroll
      for (int u = 0; u < V; u += 4)
        *reinterpret_cast<float4*>(o + i + u) =
            make_float4(Elem<T>::load(ev[u]) + Elem<T>::load(gv[u]), Elem<T>::load(ev[u + 1]) + Elem<T>::load(gv[u + 1]),
                        Elem<T>::load(ev[u + 2]) + Elem<T>::load(gv[u + 2]), Elem<T>::load(ev[u + 3]) + Elem<T>::load(gv[u + 3]));
    }
  } else {
    for (int i = threadIdx.x; i < width; i += 256) o[i] = Elem<T>::load(e[i]) + Elem<T>::load(g[i]);
  }
  if (keep) {
    __syncthreads();                                     // every thread has read the token before
    if (threadIdx.x == 0) prev[slots[b]] = tok;
  }
}

__global__ void keep_last_token_kernel(const int32_t* __restrict__ ids, const int32_t* __restrict__ take_slot,
                                       const int32_t* __restrict__ last_token, int32_t* __restrict__ prev,
                                       const int32_t* __restrict__ slots, const int32_t* __restrict__ query_start, int rows,
                                       int vocab) {
  const int b = blockIdx.x * blockDim.x + threadIdx.x;
  if (b < rows) prev[slots[b]] = token_at(ids, take_slot, last_token, query_start[b + 1] - 1, vocab);
}

}  // namespace

extern "C" int holon_bigram_embedding(const int32_t* ids, const int32_t* take_slot, const int32_t* last_token,
                                      const void* table, const void* bigram, int32_t* prev, const int32_t* slots,
                                      const int32_t* starts, const int32_t* query_start, const int32_t* token_row, float* y,
                                      int tokens, int rows, int width, int vocab, int buckets, int64_t mul_prev,
                                      int64_t mul_cur, int state_slots, int dtype, int rows_in_order, void* stream) {
  HOLON_CHECK(tokens >= 0 && rows >= 0 && width > 0 && vocab > 0 && buckets > 0 && state_slots > 0,
              "bigram_embedding: tokens=%d rows=%d width=%d vocab=%d buckets=%d", tokens, rows, width, vocab, buckets);
  HOLON_CHECK((take_slot == nullptr) == (last_token == nullptr), "bigram_embedding: slots to take from without tokens");
  HOLON_CHECK(!rows_in_order || tokens == rows, "bigram_embedding: rows in order means one token a row, got %d in %d",
              tokens, rows);
  if (tokens == 0 || rows == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
#define BIGRAM(T)                                                                                                       \
  bigram_embedding_kernel<T><<<tokens, 256, 0, s>>>(ids, take_slot, last_token, (const T*)table, (const T*)bigram, prev, \
                                                    slots, starts, query_start, token_row, y, width, vocab, buckets,     \
                                                    mul_prev, mul_cur, rows_in_order)
  if (dtype == HOLON_F32) BIGRAM(float);
  else BIGRAM(bf16_t);
#undef BIGRAM
  HOLON_LAUNCH_OK();
  if (!rows_in_order) {
    keep_last_token_kernel<<<(rows + 255) / 256, 256, 0, s>>>(ids, take_slot, last_token, prev, slots, query_start, rows,
                                                              vocab);
    HOLON_LAUNCH_OK();
  }
  return 0;
}
