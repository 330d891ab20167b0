// The state-space dual form of Mamba-2: per head a state S [N, V] with one decay a token, S <- a S + dt B x^T, and the
// read-out y = S^T C + D x. A step's rows are ranges of its flat tokens (query_start[b] .. query_start[b + 1]), each
// continuing the state in its request's slot; a row that starts at position 0 starts from zeros whatever the slot holds.
//
// Steps of single tokens: one kernel from the raw projection to y (filter, step size, recurrence). Other steps: the
// filter has run, and a row's tokens go in pieces of 256:
//   1. ssd_state_kernel   what a piece adds to the state, sum_t exp(c_end - c_t) dt_t B_t x_t^T, and its whole decay
//                         exp(c_end), c the running sum of log decays inside the piece;
//   2. ssd_walk_kernel    a row's pieces in order: the state in front of each, and the row's last state into its slot;
//   3. ssd_out_kernel     y_q = exp(c_q) S_in^T C_q + sum_{t <= q} exp(c_q - c_t) dt_t (C_q . B_t) x_t + D x_q.
// All products run on the matrix cores in float32 (v_mfma_f32_16x16x4_f32), but for C_q . B_t of bfloat16 values, which
// their bfloat16 form multiplies without loss. Running sums of log decays are formed in float64 and kept as two floats,
// so that the difference of two of them is as exact as the decay between the tokens is.
//
// v_mfma_f32_16x16x4_f32: A 16x4 (lane l: row l % 16, k = l / 16), B 4x16 (lane l: column l % 16, k = l / 16), result in
// lane l: rows 4 (l / 16) + i, i < 4, of column l % 16. Which four values of the inner dimension a product takes is free
// as long as both operands agree: product i of a group of 16 takes k = 4 (l / 16) + i, so that a result's four registers
// are the B operands of the four products over its rows, with no data movement.
#include "common.h"
#include "holon_hip.h"

typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

namespace {

constexpr int SSD_PIECE = 256, SSD_QT = 64, SSD_VG = 64;
constexpr int SSD_MAX_STATE = 256, SSD_MAX_V = 1024;

__device__ __forceinline__ float softplus_f(float z) { return z > 20.f ? z : log1pf(expf(z)); }

__device__ __forceinline__ f32x4 mfma_f32(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// -- single tokens ------------------------------------------------------------------------------------------------------
// One block a (head, row). The head's x and its group's B and C go through the filter into LDS (heads of a group each
// filter the group's B and C; the input of position p lies at place p % taps of the slot's ring, which no block of this
// step reads, so the one block that stores it need not be waited for). Thread (vq, ng) holds four neighbouring values of
// rows ng, ng + NG, ... of S; the read-out is summed over a thread's rows and then over the NG threads in order.
template <typename T, bool VEC>
__global__ void __launch_bounds__(256) ssd_step_kernel(
    const T* __restrict__ proj, int width, const T* __restrict__ conv_w, const T* __restrict__ conv_b,
    T* __restrict__ held, const float* __restrict__ dt_bias, const float* __restrict__ a_log,
    const float* __restrict__ dvec, float* __restrict__ state, float* __restrict__ y, const int32_t* __restrict__ slots,
    const int32_t* __restrict__ starts, int heads, int groups, int n, int vdim, int taps) {
  constexpr int BATCH = 8;
  __shared__ float xs[SSD_MAX_V], Bs[SSD_MAX_STATE], Cs[SSD_MAX_STATE];
  __shared__ float part[1024 + 4];
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x;
  const int per = heads / groups, g = h / per;
  const int inner = heads * vdim, gn = groups * n, channels = inner + 2 * gn;
  const int slot = slots[b], start = starts[b];
  const bool carried = start > 0;
  const T* row = proj + (int64_t)b * width;
  T* ring = held + (int64_t)slot * taps * channels;
  float* S = state + ((int64_t)slot * heads + h) * n * vdim;

  const int vq = (vdim + 3) / 4, NG = 256 / vq;
  const int mv = (tid % vq) * 4, mg = tid / vq;
  const bool active = mg < NG;
  auto load_s = [&](int r, float (&s)[4]) {
    s[0] = s[1] = s[2] = s[3] = 0.f;
    if (!carried || r >= n || !active) return;
    if constexpr (VEC) {
      const float4 f = *reinterpret_cast<const float4*>(S + (int64_t)r * vdim + mv);
      s[0] = f.x; s[1] = f.y; s[2] = f.z; s[3] = f.w;
    } else {
      for (int u = 0; u < 4; ++u) if (mv + u < vdim) s[u] = S[(int64_t)r * vdim + mv + u];
    }
  };
  float s[BATCH][4];                                     // the first rows are asked for before anything else
#pragma unroll
  for (int i = 0; i < BATCH; ++i) load_s(mg + NG * i, s[i]);

  for (int c = tid; c < vdim + 2 * n; c += 256) {
    int ch;
    if (c < vdim) ch = h * vdim + c;
    else if (c < vdim + n) ch = inner + g * n + (c - vdim);
    else ch = inner + gn + g * n + (c - vdim - n);
    const T now = row[inner + ch];
    float acc = 0.f;
    for (int j = 0; j + 1 < taps; ++j) {
      const int p = start - (taps - 1) + j;
      if (p >= 0) acc += Elem<T>::load(conv_w[(int64_t)ch * taps + j]) * Elem<T>::load(ring[(int64_t)(p % taps) * channels + ch]);
    }
    acc += Elem<T>::load(conv_w[(int64_t)ch * taps + taps - 1]) * Elem<T>::load(now);
    acc += Elem<T>::load(conv_b[ch]);
    const float v = Elem<T>::round(silu<T>(acc));
    if (c < vdim) xs[c] = v;
    else if (c < vdim + n) Bs[c - vdim] = v;
    else Cs[c - vdim - n] = v;
    if (c < vdim || h % per == 0) ring[(int64_t)(start % taps) * channels + ch] = now;
  }
  const float dt = softplus_f(Elem<T>::load(row[inner + channels + h]) + dt_bias[h]);
  const float decay = expf(-expf(a_log[h]) * dt);
  __syncthreads();
  float acc[4] = {0.f, 0.f, 0.f, 0.f}, xv[4] = {0.f, 0.f, 0.f, 0.f};
  if (active)
#pragma unroll
    for (int u = 0; u < 4; ++u) xv[u] = mv + u < vdim ? xs[mv + u] : 0.f;
  for (int r0 = mg; r0 < n && active; r0 += NG * BATCH) {
    if (r0 != mg)
#pragma unroll
      for (int i = 0; i < BATCH; ++i) load_s(r0 + NG * i, s[i]);
#pragma unroll
    for (int i = 0; i < BATCH; ++i) {
      const int r = r0 + NG * i;
      if (r >= n) break;
      const float bt = dt * Bs[r], ct = Cs[r];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        s[i][u] = decay * s[i][u] + bt * xv[u];
        acc[u] += s[i][u] * ct;
      }
      if constexpr (VEC) {
        *reinterpret_cast<float4*>(S + (int64_t)r * vdim + mv) = make_float4(s[i][0], s[i][1], s[i][2], s[i][3]);
      } else {
        for (int u = 0; u < 4; ++u) if (mv + u < vdim) S[(int64_t)r * vdim + mv + u] = s[i][u];
      }
    }
  }
  if (active)                                            // NG * vq <= 256 threads leave four values each
#pragma unroll
    for (int u = 0; u < 4; ++u) part[(mg * vq + tid % vq) * 4 + u] = acc[u];
  __syncthreads();
  for (int v = tid; v < vdim; v += 256) {
    float o = 0.f;
    for (int i = 0; i < NG; ++i) o += part[i * vq * 4 + v];
    y[(int64_t)b * inner + h * vdim + v] = o + dvec[h] * xs[v];
  }
}

// -- pieces -------------------------------------------------------------------------------------------------------------
// ROWS x COLS values from src (rows src_stride apart) into LDS rows of `pitch` values, zeros beyond rows_ok and cols, in two
// steps: `ask` sends the loads off, `put` writes what they brought (a tile's loads then travel while the tile before is
// worked on). ALIGNED: every source row starts on a 16-byte border and cols is a multiple of the vector; else `put` does it
// all, value by value.
template <typename T, typename D, int ROWS, int COLS, bool ALIGNED>
struct Tile {
  static constexpr int N = Elem<T>::kVec, PER_ROW = COLS / N, TOTAL = ROWS * PER_ROW, PER = (TOTAL + 255) / 256;
  uint4 raw[ALIGNED ? PER : 1];
  const T* src;
  int64_t src_stride;
  int rows_ok, cols;
  __device__ __forceinline__ void ask(const T* from, int64_t stride, int rows, int columns) {
    src = from; src_stride = stride; rows_ok = rows; cols = columns;
    if constexpr (ALIGNED) {
#pragma unroll
      for (int e = 0; e < PER; ++e) {
        const int idx = threadIdx.x + e * 256, r = idx / PER_ROW, c = (idx % PER_ROW) * N;
        raw[e] = make_uint4(0u, 0u, 0u, 0u);
        if (idx < TOTAL && r < rows_ok && c < cols) raw[e] = *reinterpret_cast<const uint4*>(src + r * src_stride + c);
      }
    }
  }
  __device__ __forceinline__ void put(D* dst, int pitch) const {
    if constexpr (ALIGNED) {
#pragma unroll
      for (int e = 0; e < PER; ++e) {
        const int idx = threadIdx.x + e * 256, r = idx / PER_ROW, c = (idx % PER_ROW) * N;
        if (idx >= TOTAL) continue;
        if constexpr (sizeof(D) == sizeof(T)) {
          *reinterpret_cast<uint4*>(dst + r * pitch + c) = raw[e];
        } else {
          const T* v = reinterpret_cast<const T*>(&raw[e]);
#pragma unroll
          for (int u = 0; u < N; u += 4)
            *reinterpret_cast<float4*>(dst + r * pitch + c + u) =
                make_float4(Elem<T>::load(v[u]), Elem<T>::load(v[u + 1]), Elem<T>::load(v[u + 2]), Elem<T>::load(v[u + 3]));
        }
      }
    } else {
      for (int idx = threadIdx.x; idx < ROWS * COLS; idx += 256) {
        const int r = idx / COLS, c = idx % COLS;
        const bool ok = r < rows_ok && c < cols;
        if constexpr (sizeof(D) == sizeof(T)) dst[r * pitch + c] = ok ? src[r * src_stride + c] : T(0);
        else dst[r * pitch + c] = ok ? Elem<T>::load(src[r * src_stride + c]) : 0.f;
      }
    }
  }
};

// Inclusive sum over the block's 256 threads in thread order, in float64.
__device__ __forceinline__ double scan_256(double v, double* wave_tot) {
  const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
#pragma unroll
  for (int o = 1; o < WAVE; o <<= 1) {
    const double up = __shfl_up(v, o, WAVE);
    if (lane >= o) v += up;
  }
  if (lane == WAVE - 1) wave_tot[wave] = v;
  __syncthreads();
  for (int w = 0; w < wave; ++w) v += wave_tot[w];
  return v;
}

// Grid (pieces x value groups, heads, rows). NTW: n-tiles of 16 a wave owns (state rows up to 64 NTW).
template <typename T, int NTW, bool ALIGNED>
__global__ void __launch_bounds__(256) ssd_state_kernel(
    const T* __restrict__ xbc, const T* __restrict__ dt, int64_t dt_stride, const float* __restrict__ dt_bias,
    const float* __restrict__ a_log, const int32_t* __restrict__ query_start, int tokens, int heads, int groups, int n,
    int vdim, int most, const int32_t* __restrict__ base, float* __restrict__ sums, float* __restrict__ sloc,
    float* __restrict__ decay) {
  constexpr int KT = 32, BP = 64 * NTW + 16, XP = SSD_VG + 16;    // pitches that spread four rows over the banks
  __shared__ __attribute__((aligned(16))) float Bs[KT * BP];
  __shared__ __attribute__((aligned(16))) float Xs[KT * XP];
  __shared__ float ws[SSD_PIECE];
  __shared__ double tot[4];
  __shared__ double end_s;
  const int p = blockIdx.x % most, v0 = (blockIdx.x / most) * SSD_VG, h = blockIdx.y, b = blockIdx.z, tid = threadIdx.x;
  const int lo = query_start[b] + p * SSD_PIECE, hi = min(query_start[b + 1], lo + SSD_PIECE), cnt = hi - lo;
  if (cnt <= 0) return;                                  // (the same in all of the block's threads)
  const int inner = heads * vdim, channels = inner + 2 * groups * n, g = h / (heads / groups);
  const int64_t piece = base[b] + p;
  const float step = tid < cnt ? softplus_f(Elem<T>::load(dt[(int64_t)(lo + tid) * dt_stride + h]) + dt_bias[h]) : 0.f;
  const double c = scan_256((double)(-expf(a_log[h]) * step), tot);
  if (tid == SSD_PIECE - 1) end_s = c;                   // (tokens past the piece's last add nothing)
  if (v0 == 0 && tid < cnt) {
    const int64_t at = (int64_t)h * tokens + lo + tid, plane = (int64_t)heads * tokens;
    const float chi = (float)c;
    sums[at] = step;
    sums[plane + at] = chi;
    sums[2 * plane + at] = (float)(c - (double)chi);
  }
  __syncthreads();
  ws[tid] = expf((float)(end_s - c)) * step;
  if (v0 == 0 && tid == 0) decay[piece * heads + h] = expf((float)end_s);
  __syncthreads();
  const int wave = tid / WAVE, lane = tid % WAVE, grp = lane / 16, col = lane % 16;
  f32x4 acc[NTW][4];
#pragma unroll
  for (int i = 0; i < NTW; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int vcols = min(SSD_VG, vdim - v0);
  Tile<T, float, KT, 64 * NTW, ALIGNED> bt;
  Tile<T, float, KT, SSD_VG, ALIGNED> xt;
  auto ask = [&](int t0) {
    const T* rowp = xbc + (int64_t)(lo + t0) * channels;
    bt.ask(rowp + inner + g * n, channels, cnt - t0, n);
    xt.ask(rowp + h * vdim + v0, channels, cnt - t0, vcols);
  };
  ask(0);
  for (int t0 = 0; t0 < cnt; t0 += KT) {
    bt.put(Bs, BP);
    xt.put(Xs, XP);
    __syncthreads();
    if (t0 + KT < cnt) ask(t0 + KT);
#pragma unroll
    for (int ks = 0; ks < KT / 4; ++ks) {
      const int t = ks * 4 + grp;
      const float w = ws[t0 + t];
      float xb[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) xb[j] = w * Xs[t * XP + j * 16 + col];
#pragma unroll
      for (int i = 0; i < NTW; ++i) {
        const float a = Bs[t * BP + (wave + 4 * i) * 16 + col];
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = mfma_f32(a, xb[j], acc[i][j]);
      }
    }
    __syncthreads();
  }
  float* out = sloc + (piece * heads + h) * (int64_t)n * vdim;
#pragma unroll
  for (int i = 0; i < NTW; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int nr = (wave + 4 * i) * 16 + 4 * grp + r, v = v0 + j * 16 + col;
        if (nr < n && v < vdim) out[(int64_t)nr * vdim + v] = acc[i][j][r];
      }
}

// A row's pieces in order: sloc[p] becomes the state in front of piece p; the slot takes the row's last state.
__global__ void __launch_bounds__(256) ssd_walk_kernel(float* __restrict__ state, const int32_t* __restrict__ slots,
                                                       const int32_t* __restrict__ starts,
                                                       const int32_t* __restrict__ query_start, int heads, int64_t size,
                                                       const int32_t* __restrict__ base, float* __restrict__ sloc,
                                                       const float* __restrict__ decay) {
  const int h = blockIdx.y, b = blockIdx.z;
  const int64_t e = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (e >= size) return;
  const int pieces = (query_start[b + 1] - query_start[b] + SSD_PIECE - 1) / SSD_PIECE;
  if (pieces <= 0) return;
  float* held = state + ((int64_t)slots[b] * heads + h) * size + e;
  float s = starts[b] > 0 ? *held : 0.f;
  const int64_t first = base[b];
  constexpr int AHEAD = 4;                               // pieces asked for before the first of them is used
  for (int p0 = 0; p0 < pieces; p0 += AHEAD) {
    float add[AHEAD], f[AHEAD];
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) {
      const int64_t at = (first + min(p0 + i, pieces - 1)) * heads + h;
      add[i] = sloc[at * size + e];
      f[i] = decay[at];
    }
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) {
      if (p0 + i >= pieces) break;
      sloc[((first + p0 + i) * heads + h) * size + e] = s;
      s = f[i] * s + add[i];
    }
  }
  *held = s;
}

// Grid (pieces x 4 query tiles x value groups, heads, rows). NP: state rows padded with zeros. A wave owns 16 queries
// against the group's 64 values; keys come KT at a time.
template <typename T, int NP, bool ALIGNED>
__global__ void __launch_bounds__(256) ssd_out_kernel(const T* __restrict__ xbc, const float* __restrict__ dvec,
                                                      const int32_t* __restrict__ query_start, int tokens, int heads,
                                                      int groups, int n, int vdim, int most,
                                                      const int32_t* __restrict__ base, const float* __restrict__ sums,
                                                      const float* __restrict__ sin, float* __restrict__ y) {
  constexpr bool BF = sizeof(T) == 2;
  constexpr int KT = BF ? 64 : 32;
  constexpr int CP = NP + (BF ? 8 : 4), XP = SSD_VG + 4;
  __shared__ __attribute__((aligned(16))) T Cs[SSD_QT * CP];
  __shared__ __attribute__((aligned(16))) T Bs[KT * CP];
  __shared__ __attribute__((aligned(16))) float Xs[KT * XP];
  __shared__ float dts[SSD_PIECE], chi[SSD_PIECE], clo[SSD_PIECE];
  const int tiles = most * (SSD_PIECE / SSD_QT);
  const int at = blockIdx.x % tiles, v0 = (blockIdx.x / tiles) * SSD_VG, p = at / (SSD_PIECE / SSD_QT);
  const int q0 = (at % (SSD_PIECE / SSD_QT)) * SSD_QT, h = blockIdx.y, b = blockIdx.z, tid = threadIdx.x;
  const int lo = query_start[b] + p * SSD_PIECE, hi = min(query_start[b + 1], lo + SSD_PIECE), cnt = hi - lo;
  if (q0 >= cnt) return;
  const int inner = heads * vdim, channels = inner + 2 * groups * n, g = h / (heads / groups);
  const int64_t piece = base[b] + p, plane = (int64_t)heads * tokens;
  const int vcols = min(SSD_VG, vdim - v0);
  {
    const int64_t from = (int64_t)h * tokens + lo + tid;
    const bool ok = tid < cnt;
    dts[tid] = ok ? sums[from] : 0.f;
    chi[tid] = ok ? sums[plane + from] : 0.f;
    clo[tid] = ok ? sums[2 * plane + from] : 0.f;
  }
  const bool svec = vdim % 4 == 0;
  const float* S = sin + (piece * heads + h) * (int64_t)n * vdim + v0;
  Tile<float, float, KT, SSD_VG, true> st;               // the state in front of the piece, KT rows of it at a time
  if (svec) st.ask(S, vdim, n, vcols);
  {
    Tile<T, T, SSD_QT, NP, ALIGNED> ct;
    ct.ask(xbc + (int64_t)(lo + q0) * channels + inner + groups * n + g * n, channels, cnt - q0, n);
    ct.put(Cs, CP);
  }
  Tile<T, T, KT, NP, ALIGNED> bt;
  Tile<T, float, KT, SSD_VG, ALIGNED> xt;
  auto ask = [&](int k0) {
    const T* rowp = xbc + (int64_t)(lo + k0) * channels;
    bt.ask(rowp + inner + g * n, channels, cnt - k0, n);
    xt.ask(rowp + h * vdim + v0, channels, cnt - k0, vcols);
  };
  const int wave = tid / WAVE, lane = tid % WAVE, grp = lane / 16, col = lane % 16;
  const int q = q0 + wave * 16 + col;                    // this lane's query in the piece (its column)
  f32x4 acc[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int n0 = 0; n0 < n; n0 += KT) {
    __syncthreads();
    if (svec) {
      st.put(Xs, XP);
    } else {
      Tile<float, float, KT, SSD_VG, false> one;
      one.ask(S + (int64_t)n0 * vdim, vdim, n - n0, vcols);
      one.put(Xs, XP);
    }
    __syncthreads();
    if (n0 + KT < n && svec) st.ask(S + (int64_t)(n0 + KT) * vdim, vdim, n - n0 - KT, vcols);
    if (n0 + KT >= n) ask(0);                            // the first keys travel behind the last of the state
#pragma unroll
    for (int kb = 0; kb < KT / 16; ++kb) {
      if (n0 + kb * 16 >= NP) break;
      const T* cp = Cs + (wave * 16 + col) * CP + n0 + kb * 16 + 4 * grp;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float cv = Elem<T>::load(cp[i]);
        const float* xp = Xs + (kb * 16 + 4 * grp + i) * XP + col;
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[j] = mfma_f32(xp[j * 16], cv, acc[j]);
      }
    }
  }
  const int qc = min(q, SSD_PIECE - 1);
  const float qhi = chi[qc], qlo = clo[qc];
  {
    const float f = expf(qhi + qlo);
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] *= f;
  }
  const int q_last = min(q0 + SSD_QT, cnt) - 1;          // the tile's last query
  for (int k0 = 0; k0 <= q_last; k0 += KT) {
    __syncthreads();
    bt.put(Bs, CP);
    xt.put(Xs, XP);
    __syncthreads();
    if (k0 + KT <= q_last) ask(k0 + KT);
#pragma unroll
    for (int ks = 0; ks < KT / 16; ++ks) {
      if (k0 + ks * 16 > q0 + wave * 16 + 15) break;     // keys behind every query of this wave
      f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};               // rows: keys 4 grp + i of the sixteen; column: the query
      if constexpr (BF) {
#pragma unroll
        for (int kb = 0; kb < NP / 32; ++kb) {
          const bf16x8 a = *reinterpret_cast<const bf16x8*>(Bs + (ks * 16 + col) * CP + kb * 32 + grp * 8);
          const bf16x8 c = *reinterpret_cast<const bf16x8*>(Cs + (wave * 16 + col) * CP + kb * 32 + grp * 8);
          s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, c, s, 0, 0, 0);
        }
      } else {
#pragma unroll 4
        for (int kb = 0; kb < NP / 16; ++kb) {
          const float4 a = *reinterpret_cast<const float4*>(Bs + (ks * 16 + col) * CP + kb * 16 + grp * 4);
          const float4 c = *reinterpret_cast<const float4*>(Cs + (wave * 16 + col) * CP + kb * 16 + grp * 4);
          s = mfma_f32(a.x, c.x, s);
          s = mfma_f32(a.y, c.y, s);
          s = mfma_f32(a.z, c.z, s);
          s = mfma_f32(a.w, c.w, s);
        }
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int k = k0 + ks * 16 + 4 * grp + i;
        const float f = k <= q ? expf((qhi - chi[k]) + (qlo - clo[k])) * dts[k] : 0.f;
        const float pv = s[i] * f;
        const float* xp = Xs + (ks * 16 + 4 * grp + i) * XP + col;
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[j] = mfma_f32(xp[j * 16], pv, acc[j]);
      }
    }
  }
  if (q >= cnt) return;
  const float dh = dvec[h];
  const T* xq = xbc + (int64_t)(lo + q) * channels + h * vdim;
  float* out = y + (int64_t)(lo + q) * inner + h * vdim;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int v = v0 + j * 16 + 4 * grp;
    if (svec && v < vdim) {
      *reinterpret_cast<float4*>(out + v) =
          make_float4(acc[j][0] + dh * Elem<T>::load(xq[v]), acc[j][1] + dh * Elem<T>::load(xq[v + 1]),
                      acc[j][2] + dh * Elem<T>::load(xq[v + 2]), acc[j][3] + dh * Elem<T>::load(xq[v + 3]));
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (v + i < vdim) out[v + i] = acc[j][i] + dh * Elem<T>::load(xq[v + i]);
    }
  }
}

// -- the gate and the norm behind it --------------------------------------------------------------------------------------
// One block a (part, token): u = y silu(gate), u / sqrt(mean(u^2) + eps) * weight over the part's values. REGS: a thread's
// groups of N values that stay in registers between the two passes (0: they are formed again).
template <typename T, int N, int REGS>
__global__ void __launch_bounds__(256) gated_parts_norm_kernel(const float* __restrict__ y, const T* __restrict__ gate,
                                                               int64_t gate_stride, const T* __restrict__ weight,
                                                               T* __restrict__ out, int dim, int size, float eps) {
  __shared__ float part[4];
  const int64_t t = blockIdx.y;
  const int c0 = blockIdx.x * size;
  const float* yp = y + t * dim + c0;
  const T* gp = gate + t * gate_stride + c0;
  const T* wp = weight + c0;
  T* op = out + t * dim + c0;
  auto form = [&](int i, float (&u)[N]) {
    float yv[N];
    T gv[N];
    if constexpr (N == 4) {
      const float4 f = *reinterpret_cast<const float4*>(yp + i);
      yv[0] = f.x; yv[1] = f.y; yv[2] = f.z; yv[3] = f.w;
      if constexpr (sizeof(T) == 2) *reinterpret_cast<uint2*>(gv) = *reinterpret_cast<const uint2*>(gp + i);
      else *reinterpret_cast<uint4*>(gv) = *reinterpret_cast<const uint4*>(gp + i);
    } else {
      yv[0] = yp[i];
      gv[0] = gp[i];
    }
#pragma unroll
    for (int e = 0; e < N; ++e) u[e] = yv[e] * silu<T>(Elem<T>::load(gv[e]));
  };
  auto emit = [&](int i, const float (&u)[N], float r) {
#pragma unroll
    for (int e = 0; e < N; ++e) op[i + e] = Elem<T>::store(u[e] * r * Elem<T>::load(wp[i + e]));
  };
  float held[REGS > 0 ? REGS : 1][N];
  float sq = 0.f;
  if constexpr (REGS > 0) {
#pragma unroll
    for (int k = 0; k < REGS; ++k) {
      const int i = (threadIdx.x + k * 256) * N;
      if (i < size) form(i, held[k]);
      else
#pragma unroll
        for (int e = 0; e < N; ++e) held[k][e] = 0.f;
#pragma unroll
      for (int e = 0; e < N; ++e) sq += held[k][e] * held[k][e];
    }
  } else {
    for (int i = threadIdx.x * N; i < size; i += 256 * N) {
      form(i, held[0]);
#pragma unroll
      for (int e = 0; e < N; ++e) sq += held[0][e] * held[0][e];
    }
  }
  sq = wave_sum(sq);
  if (threadIdx.x % WAVE == 0) part[threadIdx.x / WAVE] = sq;
  __syncthreads();
  const float r = 1.0f / sqrtf(((part[0] + part[1]) + (part[2] + part[3])) / (float)size + eps);
  if constexpr (REGS > 0) {
#pragma unroll
    for (int k = 0; k < REGS; ++k) {
      const int i = (threadIdx.x + k * 256) * N;
      if (i < size) emit(i, held[k], r);
    }
  } else {
    for (int i = threadIdx.x * N; i < size; i += 256 * N) {
      form(i, held[0]);
      emit(i, held[0], r);
    }
  }
}
}  // namespace

extern "C" int holon_ssd_step(const void* proj, int width, const void* conv_w, const void* conv_b, void* held,
                              const float* dt_bias, const float* a_log, const float* dvec, float* state, float* y,
                              const int32_t* slots, const int32_t* starts, int rows, int heads, int groups, int n,
                              int vdim, int taps, int state_slots, int dtype, void* stream) {
  HOLON_CHECK(rows >= 0 && rows <= 65535 && heads > 0 && groups > 0 && heads % groups == 0 && state_slots > 0,
              "ssd_step: %d rows, %d heads in %d groups", rows, heads, groups);
  HOLON_CHECK(n > 0 && n <= SSD_MAX_STATE && vdim > 0 && vdim <= SSD_MAX_V && taps >= 1 && taps <= 16,
              "ssd_step: %d state rows (at most %d), values of %d (at most %d), %d taps", n, SSD_MAX_STATE, vdim, SSD_MAX_V,
              taps);
  HOLON_CHECK(width >= 2 * heads * vdim + 2 * groups * n + heads, "ssd_step: rows of %d hold no such projection", width);
  if (rows == 0) return 0;
  const dim3 grid(heads, rows);
  hipStream_t s = (hipStream_t)stream;
#define SSD_STEP(T, V)                                                                                                \
  ssd_step_kernel<T, V><<<grid, 256, 0, s>>>((const T*)proj, width, (const T*)conv_w, (const T*)conv_b, (T*)held, dt_bias, \
                                             a_log, dvec, state, y, slots, starts, heads, groups, n, vdim, taps)
  const bool vec = vdim % 4 == 0;
  if (dtype == HOLON_F32) { if (vec) SSD_STEP(float, true); else SSD_STEP(float, false); }
  else { if (vec) SSD_STEP(bf16_t, true); else SSD_STEP(bf16_t, false); }
#undef SSD_STEP
  HOLON_LAUNCH_OK();
  return 0;
}

template <typename T, bool ALIGNED>
static void ssd_pieces(const void* xbc, const void* dt, int64_t dt_stride, const float* dt_bias, const float* a_log,
                       const float* dvec, float* state, float* y, const int32_t* slots, const int32_t* starts,
                       const int32_t* query_start, int rows, int tokens, int heads, int groups, int n, int vdim, int most,
                       const int32_t* base, float* sums, float* sloc, float* decay, hipStream_t s) {
  const int vgroups = (vdim + SSD_VG - 1) / SSD_VG;
  const dim3 grid1(most * vgroups, heads, rows);
#define SSD_STATE(NTW)                                                                                                \
  ssd_state_kernel<T, NTW, ALIGNED><<<grid1, 256, 0, s>>>((const T*)xbc, (const T*)dt, dt_stride, dt_bias, a_log,     \
                                                          query_start, tokens, heads, groups, n, vdim, most, base, sums, \
                                                          sloc, decay)
  if (n <= 64) SSD_STATE(1);
  else if (n <= 128) SSD_STATE(2);
  else SSD_STATE(4);
#undef SSD_STATE
  const int64_t size = (int64_t)n * vdim;
  ssd_walk_kernel<<<dim3((unsigned)((size + 255) / 256), heads, rows), 256, 0, s>>>(state, slots, starts, query_start, heads,
                                                                                  size, base, sloc, decay);
  const dim3 grid3(most * (SSD_PIECE / SSD_QT) * vgroups, heads, rows);
#define SSD_OUT(NP)                                                                                                  \
  ssd_out_kernel<T, NP, ALIGNED><<<grid3, 256, 0, s>>>((const T*)xbc, dvec, query_start, tokens, heads, groups, n, vdim, \
                                                       most, base, sums, sloc, y)
  if (n <= 32) SSD_OUT(32);
  else if (n <= 64) SSD_OUT(64);
  else if (n <= 128) SSD_OUT(128);
  else SSD_OUT(256);
#undef SSD_OUT
}

extern "C" int holon_ssd_scan(const void* xbc, const void* dt, int64_t dt_stride, const float* dt_bias,
                              const float* a_log, const float* dvec, float* state, float* y, const int32_t* slots,
                              const int32_t* starts, const int32_t* query_start, int rows, int tokens, int heads,
                              int groups, int n, int vdim, int state_slots, int dtype, int max_pieces,
                              const int32_t* piece_base, float* sums, float* sloc, float* decay, void* stream) {
  HOLON_CHECK(rows >= 0 && rows <= 65535 && tokens >= 0 && heads > 0 && heads <= 65535 && groups > 0 && heads % groups == 0 &&
                  state_slots > 0 && dt_stride >= heads,
              "ssd_scan: %d rows of %d tokens, %d heads in %d groups", rows, tokens, heads, groups);
  HOLON_CHECK(n > 0 && n <= SSD_MAX_STATE && vdim > 0, "ssd_scan: %d state rows (at most %d), values of %d", n, SSD_MAX_STATE,
              vdim);
  HOLON_CHECK(max_pieces > 0 && piece_base && sums && sloc && decay, "ssd_scan: rows in pieces need their table and workspace");
  if (rows == 0 || tokens == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const int vec = dtype == HOLON_F32 ? 4 : 8;
  // every tile's rows on 16-byte borders: x, B and C of a token, and the token rows themselves
  const bool aligned = vdim % vec == 0 && n % vec == 0 && (uintptr_t)xbc % 16 == 0;
#define SSD_PIECES(T, A)                                                                                              \
  ssd_pieces<T, A>(xbc, dt, dt_stride, dt_bias, a_log, dvec, state, y, slots, starts, query_start, rows, tokens, heads, \
                   groups, n, vdim, max_pieces, piece_base, sums, sloc, decay, s)
  if (dtype == HOLON_F32) { if (aligned) SSD_PIECES(float, true); else SSD_PIECES(float, false); }
  else { if (aligned) SSD_PIECES(bf16_t, true); else SSD_PIECES(bf16_t, false); }
#undef SSD_PIECES
  HOLON_LAUNCH_OK();
  return 0;
}

extern "C" int holon_gated_parts_norm(const float* y, const void* gate, int64_t gate_stride, const void* weight, void* out,
                                      int tokens, int dim, int parts, float eps, int dtype, void* stream) {
  HOLON_CHECK(tokens >= 0 && dim > 0 && parts > 0 && dim % parts == 0 && gate_stride >= dim,
              "gated_parts_norm: rows of %d in %d parts, gates %lld apart", dim, parts, (long long)gate_stride);
  hipStream_t s = (hipStream_t)stream;
  const int size = dim / parts, item = dtype == HOLON_F32 ? 4 : 2;
  const bool wide = size % 4 == 0 && (gate_stride * item) % (4 * item) == 0 && (uintptr_t)gate % (4 * item) == 0 &&
                    (uintptr_t)y % 16 == 0;
  for (int t0 = 0; t0 < tokens; t0 += 65535) {
    const dim3 grid(parts, tokens - t0 < 65535 ? tokens - t0 : 65535);
#define GPN(T, N, R)                                                                                                  \
  gated_parts_norm_kernel<T, N, R><<<grid, 256, 0, s>>>(y + (int64_t)t0 * dim, (const T*)gate + t0 * gate_stride, gate_stride, \
                                                        (const T*)weight, (T*)out + (int64_t)t0 * dim, dim, size, eps)
#define GPN_BY_SIZE(T)                                                        \
  do {                                                                        \
    if (wide && size <= 1024) GPN(T, 4, 1); else if (wide && size <= 4096) GPN(T, 4, 4); \
    else if (wide) GPN(T, 4, 0); else if (size <= 1024) GPN(T, 1, 4); else GPN(T, 1, 0); \
  } while (0)
    if (dtype == HOLON_F32) GPN_BY_SIZE(float); else GPN_BY_SIZE(bf16_t);
#undef GPN_BY_SIZE
#undef GPN
  }
  HOLON_LAUNCH_OK();
  return 0;
}
