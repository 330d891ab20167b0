// Gated linear attention: per head a state S [D, V] with a decay a key channel, S <- diag(alpha) S + k v^T, and the
// read-out after the write, o = S^T q (q times a constant). A step's rows are ranges of its flat tokens (query_start[b] ..
// query_start[b + 1]), each continuing the state in its request's slot; a row that starts at position 0 starts from zeros
// whatever the slot holds. Everything of the recurrence is float32.
//
// Steps of single tokens: one kernel from the merged projection's row to the gated, normed result (`gla_step_kernel`).
// Other steps: `gla_decay_kernel` forms the decays, and a row's tokens go in blocks of 16 through `gla_scan_kernel`:
//   p_t the product of the decays of the block's tokens up to t (t itself included), s_t of those behind t, P of all;
//   o_t = S^T (p_t q_t) + sum over j <= t of (sum_d q_t[d] k_j[d] alpha_(j+1)[d] .. alpha_t[d]) v_j
//   S  <- diag(P) S + sum_j (s_j k_j) v_j^T
// Every factor is a product of decays between two tokens and so at most 1: nothing is divided by a decay, and no
// difference of logarithms is taken. The products with S and with v run on the matrix cores in float32
// (v_mfma_f32_16x16x4_f32); the block's 16 x 16 scores are formed in vector registers, a lane carrying k_j times the
// decays since j for a few channels. Rows of more than a piece's tokens run in pieces side by side: the first pass forms
// what every piece but a row's last adds to the state, and its decays' product (`PASS` 1); `gla_walk_kernel` goes over a
// row's pieces in order; the second pass starts every piece from its true state and writes outputs.
//
// v_mfma_f32_16x16x4_f32: A 16x4 (lane l: row l % 16, k = l / 16), B 4x16 (lane l: column l % 16, k = l / 16), result in
// lane l: rows 4 (l / 16) + i, i < 4, of column l % 16. Which four values of the inner dimension a product takes is free
// as long as both operands agree: product i of a group of 16 takes k = 4 (l / 16) + i, so that a result's four registers
// are the B operands of the four products over its rows, with no data movement.
#include "common.h"
#include "holon_hip.h"

typedef float f32x4 __attribute__((ext_vector_type(4)));

namespace {

// sigmoid(z)^(1 / tau), as the exponential of the logarithm (which neither overflows nor cancels).
__device__ __forceinline__ float power_of_sigmoid(float z, float inv_tau) {
  const float log_s = fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
  return expf(log_s * inv_tau);
}

// A block takes 8 tokens and 256 channels: z = a w2 + bias with the tokens' a (columns of wider rows) shared through LDS
// and w2 transposed, [rank, channels], so that a wave's loads are contiguous and serve all 8 tokens.
constexpr int DECAY_TOKENS = 8, DECAY_MAX_RANK = 1024;
template <typename T>
__global__ void __launch_bounds__(256) gla_decay_kernel(const T* __restrict__ a, int64_t a_stride,
                                                        const T* __restrict__ w2t, const float* __restrict__ bias,
                                                        float inv_tau, float* __restrict__ y, int tokens, int channels,
                                                        int rank) {
  __shared__ float as[DECAY_TOKENS][DECAY_MAX_RANK];
  const int t0 = blockIdx.x * DECAY_TOKENS;
  const int c = blockIdx.y * 256 + threadIdx.x;
  for (int e = threadIdx.x; e < DECAY_TOKENS * rank; e += 256) {
    const int tt = e / rank, r = e - tt * rank;
    as[tt][r] = t0 + tt < tokens ? Elem<T>::load(a[(int64_t)(t0 + tt) * a_stride + r]) : 0.f;
  }
  __syncthreads();
  if (c >= channels) return;
  float acc[DECAY_TOKENS];
#pragma unroll
  for (int tt = 0; tt < DECAY_TOKENS; ++tt) acc[tt] = 0.f;
  for (int r = 0; r < rank; ++r) {
    const float wv = Elem<T>::load(w2t[(int64_t)r * channels + c]);
#pragma unroll
    for (int tt = 0; tt < DECAY_TOKENS; ++tt) acc[tt] += as[tt][r] * wv;
  }
  const float off = bias[c];
#pragma unroll
  for (int tt = 0; tt < DECAY_TOKENS; ++tt)
    if (t0 + tt < tokens) y[(int64_t)(t0 + tt) * channels + c] = power_of_sigmoid(acc[tt] + off, inv_tau);
}

struct GlaRows {
  const int32_t* slots;
  const int32_t* starts;
  const int32_t* query_start;
  int heads, dim, vdim;
  int piece;                   // tokens a piece (0: rows are not cut)
  const int32_t* base;         // [rows]: the number of row b's first piece among all pieces of the step
  float* sloc;                 // [pieces, H, D, V]: what a piece adds; after the walk, the state behind it
  float* pw;                   // [pieces, H, D]: the product of a piece's decays
};

template <int CTRL> __device__ __forceinline__ float dpp_add(float v) {
  return v + __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, false));
}

// A block: one (row or piece, head) and 16 NW value columns, wave w columns 16 w .. 16 w + 15 of them, S's KD x 16 part of
// a wave in its matrix-core accumulators. KD: the key size padded with zeros (a zero key writes nothing).
template <int KD, int NW, int PASS, typename T>
__global__ void __launch_bounds__(NW * WAVE, KD <= 64 ? 4 : 1) gla_scan_kernel(const T* __restrict__ q, const T* __restrict__ k,
                                                             const T* __restrict__ v, int64_t stride, float q_scale,
                                                             const float* __restrict__ alpha, float* __restrict__ state,
                                                             float* __restrict__ out, GlaRows r) {
  constexpr bool OUT = PASS == 2;
  constexpr int TB = 16, THREADS = NW * WAVE, N = TB * KD, PER = N / THREADS, DT = KD / 16, QP = KD + 4, TP = TB + 4;
  constexpr int VW = KD >= 16 * NW ? 4 : KD / (4 * NW), U = KD / (4 * VW * NW);      // scores: channels a lane takes at a time, times
  static_assert(N % THREADS == 0 && KD == 4 * VW * NW * U, "whole tiles");
  __shared__ __attribute__((aligned(16))) float as_[N], ks_[N], qs_[OUT ? N : 4];
  __shared__ __attribute__((aligned(16))) float qp_[OUT ? TB * QP : 4], kt_[KD * TP], P_[KD];
  __shared__ __attribute__((aligned(16))) float red_[OUT ? NW * TB * TB : 4];
  const int b = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, wave = tid / WAVE, lane = tid % WAVE;
  const int g4 = lane / 16, c = lane % 16;
  const int col_blocks = (r.vdim + 16 * NW - 1) / (16 * NW);
  const int piece = blockIdx.z / col_blocks, col0 = (blockIdx.z % col_blocks) * 16 * NW;
  const int dim = r.dim, vdim = r.vdim;
  int lo = r.query_start[b], hi = r.query_start[b + 1];
  bool from_slot = true, to_slot = OUT;
  int64_t piece_no = 0;
  if (r.piece > 0) {                                       // (everything here is the same in all of the block's lanes)
    const int pieces = (hi - lo + r.piece - 1) / r.piece;
    if (piece >= pieces || (PASS == 1 && piece == pieces - 1)) return;
    lo += piece * r.piece;
    hi = min(hi, lo + r.piece);
    from_slot = piece == 0;
    to_slot = OUT && piece == pieces - 1;
    piece_no = r.base[b] + piece;
  }
  float* held = state + ((int64_t)r.slots[b] * r.heads + h) * dim * vdim;
  const bool carried = r.starts[b] > 0;
  const int j = col0 + 16 * wave + c;                      // this lane's value column
  const bool col = j < vdim;
  f32x4 S[DT];
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * dt + 4 * g4 + i;
      const bool in = OUT && col && d < dim;
      S[dt][i] = !in ? 0.f
                     : (from_slot ? (carried ? held[(int64_t)d * vdim + j] : 0.f)
                                  : r.sloc[((piece_no - 1) * r.heads + h) * dim * vdim + (int64_t)d * vdim + j]);
    }
  float run = 1.f;                                         // PASS 1, thread d: the product of the piece's decays so far
  const int64_t width = (int64_t)r.heads * dim;
  // The operands of a block of tokens, on their way to registers as they lie in memory: places that do not exist are read
  // from ones that do and made harmless when the values are used, so that nothing here waits for a load.
  T nq[OUT ? PER : 1], nk[PER], nv[4];
  float na[PER];
  auto ask = [&](int t0) {
#pragma unroll
    for (int e = 0; e < PER; ++e) {
      const int idx = tid + e * THREADS, t = min(t0 + idx / KD, hi - 1), d = min(idx % KD, dim - 1);
      const int64_t at = (int64_t)t * stride + (int64_t)h * dim + d;
      nk[e] = k[at];
      na[e] = alpha[(int64_t)t * width + (int64_t)h * dim + d];
      if constexpr (OUT) nq[e] = q[at];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
      nv[i] = v[(int64_t)min(t0 + 4 * g4 + i, hi - 1) * stride + (int64_t)h * vdim + min(j, vdim - 1)];
  };
  if (lo < hi) ask(lo);
  for (int t0 = lo; t0 < hi; t0 += TB) {
#pragma unroll
    for (int e = 0; e < PER; ++e) {
      const int idx = tid + e * THREADS;
      const bool ok = t0 + idx / KD < hi && idx % KD < dim;
      as_[idx] = ok ? na[e] : 1.f;
      ks_[idx] = ok ? Elem<T>::load(nk[e]) : 0.f;
      if constexpr (OUT) qs_[idx] = ok ? Elem<T>::load(nq[e]) * q_scale : 0.f;
    }
    float vv[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) vv[i] = t0 + 4 * g4 + i < hi && col ? Elem<T>::load(nv[i]) : 0.f;
    lds_barrier();
    if (t0 + TB < hi) ask(t0 + TB);
    // a channel a thread: k times the decays behind each token (and all of the block's); q times those up to it
    for (int e = tid; e < (OUT ? 2 * KD : KD); e += THREADS) {
      const int d = e % KD;
      const float* src = e < KD ? ks_ : qs_;
      float a[TB], x[TB];
#pragma unroll
      for (int t = 0; t < TB; ++t) { a[t] = as_[t * KD + d]; x[t] = src[t * KD + d]; }
      if (e < KD) {
        float s = 1.f;
        f32x4 rows[TB / 4];
#pragma unroll
        for (int t = TB - 1; t >= 0; --t) {
          rows[t / 4][t % 4] = x[t] * s;
          s *= a[t];
        }
#pragma unroll
        for (int q4 = 0; q4 < TB / 4; ++q4) *reinterpret_cast<f32x4*>(&kt_[d * TP + 4 * q4]) = rows[q4];
        P_[d] = s;
        if constexpr (!OUT) run *= s;                      // (KD <= THREADS there: one channel a thread)
      } else {
        float p = 1.f;
#pragma unroll
        for (int t = 0; t < TB; ++t) {
          p *= a[t];
          qp_[t * QP + d] = x[t] * p;
        }
      }
    }
    if constexpr (OUT) {                                   // the block's scores, every wave over its channels
      typedef float fv __attribute__((ext_vector_type(VW)));
      const int jj = lane / 4, part = lane % 4;            // lane (jj, part): key jj, channels ((u NW + wave) 4 + part) VW ..
      fv kj[U], car[U];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        kj[u] = *reinterpret_cast<const fv*>(&ks_[jj * KD + ((u * NW + wave) * 4 + part) * VW]);
        car[u] = (fv)0.f;
      }
      float dot[TB];
#pragma unroll
      for (int t = 0; t < TB; ++t) {
        dot[t] = 0.f;
#pragma unroll
        for (int u = 0; u < U; ++u) {
          const int d = ((u * NW + wave) * 4 + part) * VW;
          const fv at = *reinterpret_cast<const fv*>(&as_[t * KD + d]);
          const fv qt = *reinterpret_cast<const fv*>(&qs_[t * KD + d]);
#pragma unroll
          for (int i = 0; i < VW; ++i) {
            car[u][i] = jj == t ? kj[u][i] : car[u][i] * at[i];        // (0 until the key's own token)
            dot[t] += qt[i] * car[u][i];
          }
        }
      }
#pragma unroll
      for (int t = 0; t < TB; ++t) {
        dot[t] = dpp_add<0xB1>(dot[t]);                    // quad_perm [1, 0, 3, 2]
        dot[t] = dpp_add<0x4E>(dot[t]);                    // quad_perm [2, 3, 0, 1]
      }
      if (part == 0) {
#pragma unroll
        for (int t = 0; t < TB; ++t) red_[(wave * TB + t) * TB + jj] = dot[t];
      }
    }
    lds_barrier();
    if constexpr (OUT) {
      f32x4 o[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) {
        const f32x4 qa = *reinterpret_cast<const f32x4*>(&qp_[c * QP + 16 * dt + 4 * g4]);
#pragma unroll
        for (int i = 0; i < 4; ++i) o[i % 2] = __builtin_amdgcn_mfma_f32_16x16x4f32(qa[i], S[dt][i], o[i % 2], 0, 0, 0);
      }
      f32x4 sa = *reinterpret_cast<const f32x4*>(&red_[c * TB + 4 * g4]);      // the waves' scores, added up in order
#pragma unroll
      for (int w = 1; w < NW; ++w) sa += *reinterpret_cast<const f32x4*>(&red_[(w * TB + c) * TB + 4 * g4]);
#pragma unroll
      for (int i = 0; i < 4; ++i) o[i % 2] = __builtin_amdgcn_mfma_f32_16x16x4f32(sa[i], vv[i], o[i % 2], 0, 0, 0);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = t0 + 4 * g4 + i;
        if (t < hi && col) out[((int64_t)t * r.heads + h) * vdim + j] = o[0][i] + o[1][i];
      }
    }
    if (!OUT || t0 + TB < hi || to_slot) {
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) {
        const f32x4 pd = *reinterpret_cast<const f32x4*>(&P_[16 * dt + 4 * g4]);
        const f32x4 ka = *reinterpret_cast<const f32x4*>(&kt_[(16 * dt + c) * TP + 4 * g4]);
        S[dt] *= pd;
#pragma unroll
        for (int i = 0; i < 4; ++i) S[dt] = __builtin_amdgcn_mfma_f32_16x16x4f32(ka[i], vv[i], S[dt], 0, 0, 0);
      }
    }
    // (no barrier: the next block's operands go where only the part before the last barrier read, and what this part reads
    // is written again behind the next one)
  }
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * dt + 4 * g4 + i;
      if (!col || d >= dim) continue;
      if constexpr (!OUT) r.sloc[(piece_no * r.heads + h) * dim * vdim + (int64_t)d * vdim + j] = S[dt][i];
      else if (to_slot) held[(int64_t)d * vdim + j] = S[dt][i];
    }
  if constexpr (!OUT) {
    if (col0 == 0 && tid < dim) r.pw[(piece_no * r.heads + h) * dim + tid] = run;
  }
}

// Between the passes: a row's pieces in order, S <- diag(pw) S + sloc; sloc[p] becomes the state piece p + 1 starts from.
// A thread an element; the pieces' values are asked for four at a time.
__global__ void __launch_bounds__(256) gla_walk_kernel(const float* __restrict__ state, GlaRows r) {
  const int b = blockIdx.x, h = blockIdx.y, e = blockIdx.z * 256 + threadIdx.x;
  const int cells = r.dim * r.vdim;
  if (e >= cells) return;
  const int pieces = (r.query_start[b + 1] - r.query_start[b] + r.piece - 1) / r.piece;
  const int row = e / r.vdim;
  float s = r.starts[b] > 0 ? state[((int64_t)r.slots[b] * r.heads + h) * cells + e] : 0.f;
  for (int p0 = 0; p0 + 1 < pieces; p0 += 4) {
    float add[4], w[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int64_t at = ((int64_t)r.base[b] + min(p0 + i, pieces - 2)) * r.heads + h;
      add[i] = r.sloc[at * cells + e];
      w[i] = r.pw[at * r.dim + row];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if (p0 + i + 1 >= pieces) break;
      s = w[i] * s + add[i];
      r.sloc[(((int64_t)r.base[b] + p0 + i) * r.heads + h) * cells + e] = s;
    }
  }
}

// A step of single tokens (row b is token b), from the merged projection's row to the mixer's result in front of its
// output projection: one block a (row, head). Decays, S <- diag(alpha) S + k v^T, o = S^T q, o / sqrt(mean(o^2) + eps)
// weight silu(gate). A thread holds N neighbouring columns of R rows of S (rows ty, ty + TY, ...).
template <int R, int N, typename T>
__global__ void __launch_bounds__(1024) gla_step_kernel(const T* __restrict__ q, const T* __restrict__ k,
                                                        const T* __restrict__ v, const T* __restrict__ gate,
                                                        const T* __restrict__ a, int64_t stride, float q_scale,
                                                        const T* __restrict__ w2t, const float* __restrict__ bias,
                                                        float inv_tau, int rank, const T* __restrict__ weight, float eps,
                                                        float* __restrict__ state, T* __restrict__ y,
                                                        const int32_t* __restrict__ slots,
                                                        const int32_t* __restrict__ starts, int heads, int dim, int vdim,
                                                        int tx_count, int ty_count) {
  extern __shared__ float lds[];                           // [ty_count][vdim] partial read-outs, then q, k, alpha, a
  __shared__ float part[16];
  const int b = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int tx = tid % tx_count, ty = tid / tx_count;
  const bool active = ty < ty_count;
  float* qs = lds + ty_count * vdim;
  float* ks = qs + dim;
  float* al = ks + dim;
  float* as = al + dim;
  const int j = tx * N;
  float* held = state + ((int64_t)slots[b] * heads + h) * dim * vdim;
  const bool carried = starts[b] > 0;
  float S[R][N];
#pragma unroll
  for (int i = 0; i < R; ++i) {                            // the state is asked for first: it is what takes time to come
    const int d = ty + i * ty_count;
#pragma unroll
    for (int u = 0; u < N; ++u) S[i][u] = 0.f;
    if (active && carried && d < dim && j < vdim) {
      if constexpr (N == 4) {
        const f32x4 x = *reinterpret_cast<const f32x4*>(held + (int64_t)d * vdim + j);
#pragma unroll
        for (int u = 0; u < 4; ++u) S[i][u] = x[u];
      } else {
        S[i][0] = held[(int64_t)d * vdim + j];
      }
    }
  }
  const int64_t row = (int64_t)b * stride;
  for (int e = tid; e < rank; e += blockDim.x) as[e] = Elem<T>::load(a[row + e]);
  for (int d = tid; d < dim; d += blockDim.x) {
    qs[d] = Elem<T>::load(q[row + (int64_t)h * dim + d]) * q_scale;
    ks[d] = Elem<T>::load(k[row + (int64_t)h * dim + d]);
  }
  float vt[N];
#pragma unroll
  for (int u = 0; u < N; ++u) vt[u] = j + u < vdim ? Elem<T>::load(v[row + (int64_t)h * vdim + j + u]) : 0.f;
  __syncthreads();
  const int channels = heads * dim;
  for (int d = tid; d < dim; d += blockDim.x) {
    float z = 0.f;
#pragma unroll 8
    for (int e = 0; e < rank; ++e) z += as[e] * Elem<T>::load(w2t[(int64_t)e * channels + h * dim + d]);
    al[d] = power_of_sigmoid(z + bias[h * dim + d], inv_tau);
  }
  __syncthreads();
  float o[N];
#pragma unroll
  for (int u = 0; u < N; ++u) o[u] = 0.f;
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int d = ty + i * ty_count;
    if (!active || d >= dim || j >= vdim) continue;
    const float ad = al[d], kd = ks[d], qd = qs[d];
#pragma unroll
    for (int u = 0; u < N; ++u) {
      S[i][u] = ad * S[i][u] + kd * vt[u];
      o[u] += qd * S[i][u];
    }
    if constexpr (N == 4) *reinterpret_cast<f32x4*>(held + (int64_t)d * vdim + j) = f32x4{S[i][0], S[i][1], S[i][2], S[i][3]};
    else held[(int64_t)d * vdim + j] = S[i][0];
  }
#pragma unroll
  for (int u = 0; u < N; ++u)
    if (active && j + u < vdim) lds[ty * vdim + j + u] = o[u];
  __syncthreads();
  float sum = 0.f, sq = 0.f;                               // a column a thread (vdim <= blockDim.x)
  if (tid < vdim) {
    for (int e = 0; e < ty_count; ++e) sum += lds[e * vdim + tid];
    sq = sum * sum;
  }
  sq = wave_sum(sq);
  if (tid % WAVE == 0) part[tid / WAVE] = sq;
  __syncthreads();
  if (tid >= vdim) return;
  float total = 0.f;
  for (int w = 0; w < (int)blockDim.x / WAVE; ++w) total += part[w];
  const float inv = 1.0f / sqrtf(total / (float)vdim + eps);
  const float gv = Elem<T>::load(gate[row + (int64_t)h * vdim + tid]);
  y[((int64_t)b * heads + h) * vdim + tid] = Elem<T>::store(sum * inv * Elem<T>::load(weight[tid]) * silu<T>(gv));
}

// How a single token's block is laid out: columns a thread, threads across a head's values, rows of threads, threads in
// all (whole waves; those behind the last row of threads rest), rows of S a thread; rows 0 where the kernel does not
// serve the sizes.
struct StepShape {
  int n, tx, ty, threads, rows;
};
StepShape step_shape(int dim, int vdim) {
  StepShape s{vdim % 4 == 0 ? 4 : 1, 0, 0, 0, 0};
  if (vdim > 1024) return s;                               // (a thread a column in the last part)
  s.tx = (vdim + s.n - 1) / s.n;
  s.ty = 1024 / s.tx < dim ? 1024 / s.tx : dim;
  const int need = s.ty * s.tx > vdim ? s.ty * s.tx : vdim;
  s.threads = (need + WAVE - 1) / WAVE * WAVE;
  const int rows = (dim + s.ty - 1) / s.ty;
  s.rows = rows <= 16 ? rows : 0;
  return s;
}
}  // namespace

#define BY_DTYPE(dtype, CALL)                    \
  do {                                           \
    if ((dtype) == HOLON_F32) { using T = float; CALL; } \
    else { using T = bf16_t; CALL; }             \
  } while (0)

extern "C" int holon_gla_decay(const void* a, int64_t a_stride, const void* w2t, const float* bias, float inv_tau, float* y,
                               int tokens, int channels, int rank, int dtype, void* stream) {
  HOLON_CHECK(tokens >= 0 && channels > 0 && rank > 0 && rank <= DECAY_MAX_RANK && a_stride >= rank,
              "gla_decay: %d channels, rank %d (at most %d), rows %lld apart", channels, rank, DECAY_MAX_RANK,
              (long long)a_stride);
  if (tokens == 0) return 0;
  const dim3 grid((tokens + DECAY_TOKENS - 1) / DECAY_TOKENS, (channels + 255) / 256);
  HOLON_CHECK(grid.y <= 65535, "gla_decay: %d channels exceed one launch", channels);
  BY_DTYPE(dtype, (gla_decay_kernel<T><<<grid, 256, 0, (hipStream_t)stream>>>((const T*)a, a_stride, (const T*)w2t, bias,
                                                                              inv_tau, y, tokens, channels, rank)));
  HOLON_LAUNCH_OK();
  return 0;
}

template <int KD, int NW, typename T>
static void launch_gla(int pass, dim3 grid, hipStream_t s, const void* q, const void* k, const void* v, int64_t stride,
                       float q_scale, const float* alpha, float* state, float* out, GlaRows r) {
  if (pass == 1)
    gla_scan_kernel<KD, NW, 1, T><<<grid, NW * WAVE, 0, s>>>((const T*)q, (const T*)k, (const T*)v, stride, q_scale, alpha,
                                                             state, out, r);
  else
    gla_scan_kernel<KD, NW, 2, T><<<grid, NW * WAVE, 0, s>>>((const T*)q, (const T*)k, (const T*)v, stride, q_scale, alpha,
                                                             state, out, r);
}

extern "C" int holon_gla_scan(const void* q, const void* k, const void* v, int64_t stride, float q_scale, const float* alpha,
                              float* state, float* out, const int32_t* slots, const int32_t* starts,
                              const int32_t* query_start, int rows, int heads, int dim, int vdim, int state_slots,
                              int dtype, int piece_tokens, int max_pieces, const int32_t* piece_base, float* sloc,
                              float* pw, void* stream) {
  HOLON_CHECK(rows >= 0 && heads > 0 && heads <= 65535 && dim > 0 && dim <= 256 && vdim > 0 && state_slots > 0,
              "gla_scan: %d heads of %d (at most 256) by %d", heads, dim, vdim);
  HOLON_CHECK(stride >= (int64_t)heads * dim && stride >= (int64_t)heads * vdim, "gla_scan: rows %lld apart for %d heads",
              (long long)stride, heads);
  HOLON_CHECK(piece_tokens == 0 || (piece_tokens > 0 && piece_tokens % 16 == 0 && max_pieces > 0 && piece_base && sloc && pw),
              "gla_scan: rows in pieces of %d tokens (a multiple of 16) need the pieces' table and workspace", piece_tokens);
  if (rows == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const GlaRows r{slots, starts, query_start, heads, dim, vdim, piece_tokens, piece_base, sloc, pw};
  const int nw = vdim <= 64 ? 4 : 8;
  const int col_blocks = (vdim + 16 * nw - 1) / (16 * nw);
  const int most = piece_tokens ? max_pieces : 1;
  HOLON_CHECK((int64_t)col_blocks * most <= 65535 && ((int64_t)dim * vdim + 255) / 256 <= 65535,
              "gla_scan: %d pieces of %d x %d exceed one launch", most, dim, vdim);
  const dim3 grid(rows, heads, col_blocks * most);
#define GLA_NW(PASS, KD)                                                                                              \
  do {                                                                                                                \
    if (nw == 4) launch_gla<KD, 4, T>(PASS, grid, s, q, k, v, stride, q_scale, alpha, state, out, r);                  \
    else launch_gla<KD, 8, T>(PASS, grid, s, q, k, v, stride, q_scale, alpha, state, out, r);                          \
  } while (0)
#define GLA(PASS)                                                                                                     \
  do {                                                                                                                \
    if (dim <= 32) BY_DTYPE(dtype, GLA_NW(PASS, 32));                                                                  \
    else if (dim <= 64) BY_DTYPE(dtype, GLA_NW(PASS, 64));                                                             \
    else if (dim <= 128) BY_DTYPE(dtype, GLA_NW(PASS, 128));                                                           \
    else BY_DTYPE(dtype, GLA_NW(PASS, 256));                                                                           \
  } while (0)
  if (piece_tokens) {
    GLA(1);
    HOLON_LAUNCH_OK();
    gla_walk_kernel<<<dim3(rows, heads, (dim * vdim + 255) / 256), 256, 0, s>>>(state, r);
    HOLON_LAUNCH_OK();
  }
  GLA(2);
#undef GLA
#undef GLA_NW
  HOLON_LAUNCH_OK();
  return 0;
}

extern "C" int holon_gla_step_supported(int dim, int vdim) {
  return dim > 0 && dim <= 256 && vdim > 0 && step_shape(dim, vdim).rows > 0;
}

extern "C" int holon_gla_step(const void* q, const void* k, const void* v, const void* gate, const void* a, int64_t stride,
                              float q_scale, const void* w2t, const float* bias, float inv_tau, int rank,
                              const void* weight, float eps, float* state, void* y, const int32_t* slots,
                              const int32_t* starts, int rows, int heads, int dim, int vdim, int state_slots, int dtype,
                              void* stream) {
  HOLON_CHECK(rows >= 0 && heads > 0 && heads <= 65535 && rank > 0 && rank <= DECAY_MAX_RANK && state_slots > 0 &&
                  holon_gla_step_supported(dim, vdim),
              "gla_step: %d heads of %d by %d, rank %d", heads, dim, vdim, rank);
  HOLON_CHECK(stride >= (int64_t)heads * dim && stride >= (int64_t)heads * vdim && (uintptr_t)state % 16 == 0,
              "gla_step: rows %lld apart for %d heads", (long long)stride, heads);
  if (rows == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const StepShape sh = step_shape(dim, vdim);
  const size_t lds = ((size_t)sh.ty * vdim + 3 * (size_t)dim + rank) * sizeof(float);
  const dim3 grid(rows, heads);
#define STEP(R, N)                                                                                                     \
  BY_DTYPE(dtype, (gla_step_kernel<R, N, T><<<grid, sh.threads, lds, s>>>(                                              \
                      (const T*)q, (const T*)k, (const T*)v, (const T*)gate, (const T*)a, stride, q_scale, (const T*)w2t, \
                      bias, inv_tau, rank, (const T*)weight, eps, state, (T*)y, slots, starts, heads, dim, vdim, sh.tx, sh.ty)))
#define STEP_N(R) do { if (sh.n == 4) STEP(R, 4); else STEP(R, 1); } while (0)
  if (sh.rows <= 1) STEP_N(1);
  else if (sh.rows <= 2) STEP_N(2);
  else if (sh.rows <= 4) STEP_N(4);
  else if (sh.rows <= 8) STEP_N(8);
  else STEP_N(16);
#undef STEP_N
#undef STEP
  HOLON_LAUNCH_OK();
  return 0;
}
