// Time mixing with a token shift and a state whose decay is computed from the token, with a bonus for the current token.
//
// A step is a flattened batch: token t belongs to request token_request[t], whose new tokens are rows
// cu_q[b] .. cu_q[b+1]-1 and whose states are rows state_slots[b] of the state tensors. Decays with their
// exponentials, the state and every sum into it, head norms and gates are float32 in either precision.
#include "common.h"
#include "vector_values.h"

namespace {

constexpr int SHIFT_MAX_MIXES = 8;

// out[k][t] = x_t + (x_(t-1) - x_t) * mu[k] for every mix k; the row before a request's first row of the step is its
// state row. The thread that reads a state value is the one that replaces it by the request's last row of the step.
template <int V, typename X>
__global__ void token_shift_kernel(const X* __restrict__ x, const float* __restrict__ mu, int mixes, float* __restrict__ state,
                                   X* __restrict__ out, const int32_t* __restrict__ cu_q,
                                   const int32_t* __restrict__ token_request, const int32_t* __restrict__ state_slots, int C,
                                   int64_t T) {
  const int64_t t = blockIdx.x;
  const int c = V * static_cast<int>(blockIdx.y * blockDim.x + threadIdx.x);
  if (c >= C) return;
  const int b = token_request != nullptr ? token_request[t] : static_cast<int>(t);     // null: a row a request
  const int64_t first = token_request != nullptr ? cu_q[b] : t;
  float h[V], before[V];
  load_values<V>(x + t * C + c, h);
  if (t > first) {
    load_values<V>(x + (t - 1) * C + c, before);
  } else {
    float* own = state + static_cast<int64_t>(state_slots[b]) * C + c;
    const int64_t last = token_request != nullptr ? cu_q[b + 1] - 1 : t;
    float keep[V];
    load_values<V>(own, before);
    load_values<V>(x + last * C + c, keep);
    store_values<V>(own, keep);
  }
#pragma unroll
  for (int k = 0; k < V; ++k) before[k] -= h[k];
  for (int m = 0; m < mixes; ++m) {
    float w[V], v[V];
    load_values<V>(mu + static_cast<int64_t>(m) * C + c, w);
#pragma unroll
    for (int k = 0; k < V; ++k) v[k] = h[k] + before[k] * w[k];
    store_values<V>(out + (m * T + t) * C + c, v);
  }
}

// ---------------------------------------------------------------------------------------------------
// Row after row. A block owns one head of one request: thread (part, e) keeps rows d = part, part + PARTS, ... of column e
// of the state in registers. Per token: the decay of every key channel from `low` (tanh, the second projection, both
// exponentials; `z` instead of `low` where the projection was made before), then
//   o[e] = sum_d r[d] (S[d][e] + u[d] k[d] v[e]);   S[d][e] = w[d] S[d][e] + k[d] v[e]
// the PARTS partial sums of a column meet in LDS, the head's norm is taken over its D columns, times its weight and
// silu(gate). The next token's values are asked for before this token's are used.
template <typename X, typename L, typename O, int COLS, int PARTS, int ROWS>
__global__ void __launch_bounds__(COLS * PARTS)
wkv_scan_kernel(const X* __restrict__ r_in, const X* __restrict__ k_in, const X* __restrict__ v_in,
                const X* __restrict__ gates, int64_t ld, const L* __restrict__ low, int64_t ld_low, int rank,
                const float* __restrict__ up, const float* __restrict__ up_bias, const float* __restrict__ bonus,
                float* __restrict__ state, const float* __restrict__ norm_weight, float eps, O* __restrict__ out,
                const int32_t* __restrict__ cu_q, const int32_t* __restrict__ state_slots, int H, int D) {
  extern __shared__ float low_s[];                         // [rank]
  __shared__ float r_s[PARTS * ROWS], k_s[PARTS * ROWS], w_s[PARTS * ROWS], u_s[PARTS * ROWS];
  __shared__ float partial[PARTS][COLS];
  __shared__ float squares[COLS / 64];
  constexpr int THREADS = COLS * PARTS;
  constexpr int SUB = THREADS / (PARTS * ROWS);            // threads that share a channel's decay (4 at least, a power of two)
  const int b = blockIdx.x, head = blockIdx.y;
  const int e = threadIdx.x % COLS, part = threadIdx.x / COLS;
  const int first = cu_q != nullptr ? cu_q[b] : b, last = cu_q != nullptr ? cu_q[b + 1] : b + 1;     // null: a row a request
  if (first >= last) return;
  float* own = state + (static_cast<int64_t>(state_slots[b]) * H + head) * D * D;
  float s[ROWS];
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int d = part + i * PARTS;
    s[i] = (d < D && e < D) ? own[static_cast<int64_t>(d) * D + e] : 0.f;
  }
  const int d_own = threadIdx.x;                           // the channel whose r and k this thread fetches
  const int channel = threadIdx.x / SUB, sub = threadIdx.x % SUB;      // the channel whose decay it helps to make
  const float* up_row = up + static_cast<int64_t>(head * D + min(channel, D - 1)) * rank;
  const float z0 = up_bias[head * D + min(channel, D - 1)];
  constexpr int UP_HELD = 16;                              // of the channel's row, kept for all tokens
  float up_held[UP_HELD];
#pragma unroll
  for (int i = 0; i < UP_HELD; ++i) up_held[i] = sub + i * SUB < rank ? up_row[sub + i * SUB] : 0.f;
  if (d_own < D) u_s[d_own] = bonus[head * D + d_own];
  const float weight = e < D ? norm_weight[head * D + e] : 0.f;
  float nr = 0.f, nk = 0.f, nv = 0.f, ng = 0.f, nl = 0.f;
  auto fetch = [&](int t) {
    const int64_t row = static_cast<int64_t>(t) * ld + head * D;
    if (d_own < D) nr = to_float(r_in[row + d_own]), nk = to_float(k_in[row + d_own]);
    if (e < D) nv = to_float(v_in[row + e]), ng = to_float(gates[row + e]);
    if (threadIdx.x < rank) nl = to_float(low[static_cast<int64_t>(t) * ld_low + threadIdx.x]);
  };
  fetch(first);
  for (int t = first; t < last; ++t) {
    if (threadIdx.x < rank) low_s[threadIdx.x] = tanhf(nl);
    for (int i = threadIdx.x + THREADS; i < rank; i += THREADS)
      low_s[i] = tanhf(to_float(low[static_cast<int64_t>(t) * ld_low + i]));
    if (d_own < D) r_s[d_own] = nr, k_s[d_own] = nk;
    const float v = nv, g = ng;
    if (t + 1 < last) fetch(t + 1);
    __syncthreads();
    float z = 0.f;
#pragma unroll
    for (int i = 0; i < UP_HELD; ++i) z += up_held[i] * (sub + i * SUB < rank ? low_s[sub + i * SUB] : 0.f);
    for (int i = sub + UP_HELD * SUB; i < rank; i += SUB) z += up_row[i] * low_s[i];
#pragma unroll
    for (int o = SUB / 2; o > 0; o >>= 1) z += __shfl_xor(z, o, 64);
    if (sub == 0 && channel < D) w_s[channel] = expf(-expf(z + z0));
    __syncthreads();
    float o = 0.f;
#pragma unroll
    for (int i = 0; i < ROWS; ++i) {
      const int d = part + i * PARTS;
      if (d < D) {
        const float kv = k_s[d] * v;
        o += r_s[d] * (s[i] + u_s[d] * kv);
        s[i] = w_s[d] * s[i] + kv;
      }
    }
    partial[part][e] = o;
    __syncthreads();
    float total = 0.f;
#pragma unroll
    for (int p = 0; p < PARTS; ++p) total += partial[p][e];
    float sq = wave_sum(e < D ? total * total : 0.f);
    if constexpr (COLS > 64) {
      if (part == 0 && e % 64 == 0) squares[e / 64] = sq;
      __syncthreads();
      sq = 0.f;
#pragma unroll
      for (int i = 0; i < COLS / 64; ++i) sq += squares[i];
    }
    if (part == 0 && e < D)
      out[(static_cast<int64_t>(t) * H + head) * D + e] =
          from_float<O>(total / sqrtf(sq / D + eps) * weight * (g / (1.f + expf(-g))));
    // (the next token's values go to other places of LDS than what is read behind the last barrier, but for the
    // partial sums and the squares, which two barriers stand in front of)
  }
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int d = part + i * PARTS;
    if (d < D && e < D) own[static_cast<int64_t>(d) * D + e] = s[i];
  }
}

// ---------------------------------------------------------------------------------------------------
// The same recurrence over portions of prompts, in chunks of 64 rows that run side by side. With S the state in front of
// a chunk and c_i the sum of ln w over its rows up to and with i:
//   sums:     P[d][e] = sum_j exp(c_L[d] - c_j[d]) k_j[d] v_j[e],   G[d] = exp(c_L[d])            (each chunk alone)
//   states:   S_next = diag(G) S + P, chunk after chunk; the state in front of a chunk takes P's place
//   outputs:  o_i[e] = sum_d r_i[d] exp(c_(i-1)[d]) S[d][e] + sum_(j < i) (sum_d r_i[d] k_j[d] exp(c_(i-1)[d] - c_j[d])) v_j[e]
//                      + (sum_d r_i[d] u[d] k_i[d]) v_i[e]
// and behind them head norm, weight and gate. Everything is float32, the tiles' products on v_mfma_f32_16x16x4_f32.
//
// A chunk is four runs of 16 rows, a wave each. A wave's lane (i = lane % 16, g = lane / 16) owns row i of the run and the
// channels DL g .. DL g + DL - 1 (DL = DP / 4) of r, k and ln w: the matrix cores' operand with the summed index in an order
// of our own. Sums of ln w run over the rows of one run only, by row shifts between the lanes; what lies between two runs
// enters as a product of the runs' total factors. So every exponent is <= 0, no quotient of decays is formed, and differences
// are taken over 16 rows at most. The scores between different runs are products of the matrix cores, taken transposed:
// their result lies as the next product's operand. Those within a run need an exponential of their own for every pair and
// channel: row j of k and ln w goes to all lanes of its group by a row broadcast.
constexpr int WK_ROWS = 64;
constexpr float LOG2E = 1.4426950408889634f;

typedef __attribute__((__vector_size__(4 * sizeof(float)))) float floatx4;

template <int CTRL>
__device__ __forceinline__ float row_move(float x) {          // a DPP move within rows of 16 lanes; 0 where nothing comes in
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, x), CTRL, 0xf, 0xf, true));
}
template <int N>
__device__ __forceinline__ float row_shift(float x) { return row_move<0x110 + N>(x); }       // from the lane N below
template <int N>
__device__ __forceinline__ float row_lane(float x) { return row_move<0x150 + N>(x); }        // lane N of the row, to all

__device__ __forceinline__ float groups_sum(float v) {        // over the four lanes that own a row
  v += __shfl_xor(v, 16, 64);
  return v + __shfl_xor(v, 32, 64);
}

// a lane's channels of one row of a head (`row` points at the head's first column); zeros for a row that is not there
template <int DP, typename X>
__device__ __forceinline__ void load_channels(const X* __restrict__ row, int D, int g, bool there, bool whole, float out[DP / 4]) {
  constexpr int DL = DP / 4;
#pragma unroll
  for (int s = 0; s < DL; ++s) out[s] = 0.f;
  if (!there) return;
  if (whole) {
#pragma unroll
    for (int s = 0; s < DL; s += 4) load_values<4>(row + DL * g + s, out + s);
  } else {
#pragma unroll
    for (int s = 0; s < DL; ++s)
      if (DL * g + s < D) out[s] = to_float(row[DL * g + s]);
  }
}

// log2 of the decays of a lane's channels, summed over the rows of the run up to the lane's own
template <int DP>
__device__ __forceinline__ void run_decays(const float* __restrict__ z, int D, int g, bool there, bool whole, float c[DP / 4]) {
  constexpr int DL = DP / 4;
  load_channels<DP>(z, D, g, there, whole, c);
#pragma unroll
  for (int s = 0; s < DL; ++s) {
    // (a factor of 2^-160 is zero in float32: smaller ones need no larger exponents, and infinities have no differences)
    c[s] = there ? fmaxf(-LOG2E * expf(c[s]), -160.f) : 0.f;
    c[s] += row_shift<1>(c[s]);
    c[s] += row_shift<2>(c[s]);
    c[s] += row_shift<4>(c[s]);
    c[s] += row_shift<8>(c[s]);
  }
}

// V of a chunk into LDS as float32, rows DP + 4 apart, zeros for what is not there
template <int DP, typename X>
__device__ __forceinline__ void stage_rows(const X* __restrict__ v, int64_t ld, int len, int D, bool whole, float* __restrict__ to) {
  constexpr int RUNS = DP / 4;
  for (int idx = threadIdx.x; idx < WK_ROWS * RUNS; idx += blockDim.x) {
    const int j = idx / RUNS, e = idx % RUNS * 4;
    float x[4] = {};
    if (j < len) {
      if (whole) {
        load_values<4>(v + j * ld + e, x);
      } else {
#pragma unroll
        for (int k = 0; k < 4; ++k)
          if (e + k < D) x[k] = to_float(v[j * ld + e + k]);
      }
    }
    store_values<4>(to + j * (DP + 4) + e, x);
  }
}

template <int DP, typename X>
__global__ void __launch_bounds__(256)
wkv_chunk_sums_kernel(const X* __restrict__ k_in, const X* __restrict__ v_in, int64_t ld, const float* __restrict__ z,
                      float* __restrict__ scratch, float* __restrict__ totals, const int4* __restrict__ chunks, int H, int D,
                      int whole) {
  constexpr int DL = DP / 4, STRIDE = DP + 4;
  __shared__ __attribute__((aligned(16))) float Ks[WK_ROWS * STRIDE];
  __shared__ __attribute__((aligned(16))) float Vs[WK_ROWS * STRIDE];
  __shared__ float factor[4][DP];
  const int head = blockIdx.y;
  const int4 chunk = chunks[blockIdx.x];
  const int64_t row0 = chunk.y;
  const int len = chunk.z;
  const int lane = threadIdx.x % 64, run = threadIdx.x / 64, i = lane % 16, g = lane / 16;
  const int row = 16 * run + i;
  float k[DL], c[DL];
  load_channels<DP>(k_in + (row0 + row) * ld + head * D, D, g, row < len, whole, k);
  run_decays<DP>(z + ((row0 + row) * H + head) * D, D, g, row < len, whole, c);
  stage_rows<DP>(v_in + row0 * ld + head * D, ld, len, D, whole, Vs);
#pragma unroll
  for (int s = 0; s < DL; ++s) {
    const float total = row_lane<15>(c[s]);
    k[s] *= __builtin_amdgcn_exp2f(total - c[s]);
    if (i == 0) factor[run][DL * g + s] = __builtin_amdgcn_exp2f(total);
  }
  __syncthreads();
  for (int later = run + 1; later < 4; ++later) {
#pragma unroll
    for (int s = 0; s < DL; ++s) k[s] *= factor[later][DL * g + s];
  }
#pragma unroll
  for (int s = 0; s < DL; s += 4) store_values<4>(Ks + row * STRIDE + DL * g + s, k + s);
  if (threadIdx.x < D)
    totals[(static_cast<int64_t>(blockIdx.x) * H + head) * D + threadIdx.x] =
        factor[0][threadIdx.x] * factor[1][threadIdx.x] * factor[2][threadIdx.x] * factor[3][threadIdx.x];
  __syncthreads();
  float* dst = scratch + (static_cast<int64_t>(blockIdx.x) * H + head) * D * D;
  for (int tile = run; tile < DP / 16; tile += 4) {
    floatx4 acc[DP / 16];
#pragma unroll
    for (int e = 0; e < DP / 16; ++e) acc[e] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int m = 0; m < 4; ++m)
#pragma unroll
      for (int s = 0; s < 4; ++s) {
        const int at = (16 * m + 4 * g + s) * STRIDE + i;
        const float a = Ks[at + 16 * tile];
#pragma unroll
        for (int e = 0; e < DP / 16; ++e) acc[e] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, Vs[at + 16 * e], acc[e], 0, 0, 0);
      }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 16 * tile + 4 * g + r;
      if (d >= D) continue;
#pragma unroll
      for (int e = 0; e < DP / 16; ++e)
        if (16 * e + i < D) dst[static_cast<int64_t>(d) * D + 16 * e + i] = acc[e][r];
    }
  }
}

__global__ void wkv_chunk_states_kernel(float* __restrict__ scratch, const float* __restrict__ totals,
                                        float* __restrict__ state, const int32_t* __restrict__ request_chunks,
                                        const int32_t* __restrict__ state_slots, int H, int D) {
  const int b = blockIdx.x, head = blockIdx.y;
  const int idx = blockIdx.z * blockDim.x + threadIdx.x;
  if (idx >= D * D) return;
  const int c0 = request_chunks[b], c1 = request_chunks[b + 1];
  if (c0 >= c1) return;
  float* own = state + (static_cast<int64_t>(state_slots[b]) * H + head) * D * D + idx;
  const int64_t stride = static_cast<int64_t>(H) * D * D;
  float* p = scratch + (static_cast<int64_t>(c0) * H + head) * D * D + idx;
  const float* factor = totals + (static_cast<int64_t>(c0) * H + head) * D + idx / D;
  float S = *own;
  for (int c = c0; c < c1; c += 8) {
    // the sums of eight chunks are asked for together; each then gives way to the state in front of its chunk
    float add[8], keep[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      const int at = min(u, c1 - 1 - c);
      add[u] = p[at * stride];
      keep[u] = factor[static_cast<int64_t>(at) * H * D];
    }
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      if (c + u >= c1) break;
      p[u * stride] = S;
      S = keep[u] * S + add[u];
    }
    p += 8 * stride;
    factor += 8 * static_cast<int64_t>(H) * D;
  }
  *own = S;
}

// the scores of a run's rows against its own row J, for one J after the other: lane (i, g) gets column 4 g + s in `a[s]`
template <int J, int DP>
__device__ __forceinline__ void run_scores(const float r[DP / 4], const float k[DP / 4], const float x[DP / 4],
                                           const float c[DP / 4], int i, int g, float a[4]) {
  if constexpr (J < 15) {
    float sum = 0.f;
#pragma unroll
    for (int s = 0; s < DP / 4; ++s) sum += r[s] * row_lane<J>(k[s]) * __builtin_amdgcn_exp2f(fminf(x[s] - row_lane<J>(c[s]), 0.f));
    sum = groups_sum(sum);
    if (g == J / 4) a[J % 4] = i > J ? sum : 0.f;
    run_scores<J + 1, DP>(r, k, x, c, i, g, a);
  }
}

template <int DP, typename X, typename O>
__global__ void __launch_bounds__(256)
wkv_chunk_outputs_kernel(const X* __restrict__ r_in, const X* __restrict__ k_in, const X* __restrict__ v_in,
                         const X* __restrict__ gates, int64_t ld, const float* __restrict__ z, const float* __restrict__ bonus,
                         const float* __restrict__ scratch, const float* __restrict__ norm_weight, float eps,
                         O* __restrict__ out, const int4* __restrict__ chunks, int H, int D, int whole) {
  constexpr int DL = DP / 4, STRIDE = DP + 4;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* Vs = lds;                                  // [64][DP + 4]
  float* Ss = Vs + WK_ROWS * STRIDE;                // [DP][DP], the columns of row d turned by 16 (d / DL) places
  float* Kt = Ss + DP * DP;                         // [4 runs][DL / 4][64 lanes][4]: k_j exp(the run's decay behind j)
  float* factor = Kt + WK_ROWS * DP;                // [4][DP]: the runs' total factors
  const int head = blockIdx.y;
  const int4 chunk = chunks[blockIdx.x];
  const int64_t row0 = chunk.y;
  const int len = chunk.z;
  const int lane = threadIdx.x % 64, run = threadIdx.x / 64, i = lane % 16, g = lane / 16;
  const int row = 16 * run + i;
  float r[DL], k[DL], c[DL], x[DL];
  load_channels<DP>(r_in + (row0 + row) * ld + head * D, D, g, row < len, whole, r);
  load_channels<DP>(k_in + (row0 + row) * ld + head * D, D, g, row < len, whole, k);
  run_decays<DP>(z + ((row0 + row) * H + head) * D, D, g, row < len, whole, c);
  stage_rows<DP>(v_in + row0 * ld + head * D, ld, len, D, whole, Vs);
  const float* src = scratch + (static_cast<int64_t>(blockIdx.x) * H + head) * D * D;
  for (int idx = threadIdx.x; idx < DP * DP / 4; idx += blockDim.x) {
    const int d = idx / (DP / 4), e = idx % (DP / 4) * 4;
    float v[4] = {};
    if (whole) {
      load_values<4>(src + static_cast<int64_t>(d) * D + e, v);
    } else if (d < D) {
#pragma unroll
      for (int q = 0; q < 4; ++q)
        if (e + q < D) v[q] = src[static_cast<int64_t>(d) * D + e + q];
    }
    store_values<4>(Ss + d * DP + (e + 16 * (d / DL)) % DP, v);
  }
#pragma unroll
  for (int s = 0; s < DL; s += 4) {
    float kt[4];
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const float total = row_lane<15>(c[s + q]);
      kt[q] = k[s + q] * __builtin_amdgcn_exp2f(total - c[s + q]);
      if (i == 0) factor[run * DP + DL * g + s + q] = __builtin_amdgcn_exp2f(total);
    }
    store_values<4>(Kt + ((run * (DL / 4) + s / 4) * 64 + lane) * 4, kt);
  }
  float own = 0.f;
#pragma unroll
  for (int s = 0; s < DL; ++s) {
    x[s] = row_shift<1>(c[s]);
    own += DL * g + s < D ? r[s] * bonus[head * D + DL * g + s] * k[s] : 0.f;
  }
  own = groups_sum(own);
  float a[4] = {};
  run_scores<0, DP>(r, k, x, c, i, g, a);
#pragma unroll
  for (int s = 0; s < 4; ++s)
    if (4 * g + s == i) a[s] = own;
#pragma unroll
  for (int s = 0; s < DL; ++s) r[s] *= __builtin_amdgcn_exp2f(x[s]);
  __syncthreads();
  floatx4 acc[DP / 16];
#pragma unroll
  for (int e = 0; e < DP / 16; ++e) acc[e] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int s = 0; s < 4; ++s)
#pragma unroll
    for (int e = 0; e < DP / 16; ++e)
      acc[e] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[s], Vs[(16 * run + 4 * g + s) * STRIDE + 16 * e + i], acc[e], 0, 0, 0);
  for (int before = run - 1; before >= 0; --before) {
    floatx4 scores = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < DL; s += 4) {
      float kt[4];
      load_values<4>(Kt + ((before * (DL / 4) + s / 4) * 64 + lane) * 4, kt);
#pragma unroll
      for (int q = 0; q < 4; ++q) scores = __builtin_amdgcn_mfma_f32_16x16x4f32(kt[q], r[s + q], scores, 0, 0, 0);
    }
#pragma unroll
    for (int s = 0; s < 4; ++s)
#pragma unroll
      for (int e = 0; e < DP / 16; ++e)
        acc[e] = __builtin_amdgcn_mfma_f32_16x16x4f32(scores[s], Vs[(16 * before + 4 * g + s) * STRIDE + 16 * e + i], acc[e], 0, 0, 0);
#pragma unroll
    for (int s = 0; s < DL; ++s) r[s] *= factor[before * DP + DL * g + s];
  }
#pragma unroll
  for (int s = 0; s < DL; ++s)
#pragma unroll
    for (int e = 0; e < DP / 16; ++e)
      acc[e] = __builtin_amdgcn_mfma_f32_16x16x4f32(r[s], Ss[(DL * g + s) * DP + (16 * e + i + 16 * g) % DP], acc[e], 0, 0, 0);
  // lane (i, g) now holds rows 4 g .. 4 g + 3 of the run, column i of every 16
#pragma unroll
  for (int q = 0; q < 4; ++q) {
    float sq = 0.f;
#pragma unroll
    for (int e = 0; e < DP / 16; ++e) sq += acc[e][q] * acc[e][q];
#pragma unroll
    for (int o = 8; o > 0; o >>= 1) sq += __shfl_xor(sq, o, 64);
    const float scale = 1.f / sqrtf(sq / D + eps);
    const int at = 16 * run + 4 * g + q;
    if (at >= len) continue;
    const int64_t t = row0 + at;
#pragma unroll
    for (int e = 0; e < DP / 16; ++e) {
      const int col = 16 * e + i;
      if (col >= D) continue;
      const float gate = to_float(gates[t * ld + head * D + col]);
      out[(t * H + head) * D + col] =
          from_float<O>(acc[e][q] * scale * norm_weight[head * D + col] * (gate / (1.f + expf(-gate))));
    }
  }
}

__global__ void tanh_f32_kernel(const float* __restrict__ in, int64_t ld, float* __restrict__ out, int N, int64_t T) {
  const int64_t i = static_cast<int64_t>(blockIdx.x) * blockDim.x + threadIdx.x;
  if (i >= T * N) return;
  out[i] = tanhf(in[i / N * ld + i % N]);
}

}  // namespace

extern "C" int distie_token_shift(const void* x, int dtype, const float* mu, int mixes, float* state, void* out,
                                  const int32_t* cu_q, const int32_t* token_request, const int32_t* state_slots, int T, int C,
                                  hipStream_t stream) {
  if (T <= 0) return 0;
  if (C < 1 || mixes < 1 || mixes > SHIFT_MAX_MIXES) return DISTIE_BAD_ARGUMENT;
  const auto aligned = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  const bool wide = C % 8 == 0 && aligned(x) && aligned(mu) && aligned(state) && aligned(out);
  const int runs = wide ? C / 8 : C;
  const int threads = runs >= 256 ? 256 : (runs > 64 ? 128 : 64);
  const dim3 grid(T, (runs + threads - 1) / threads);
  if (wide) {
    DISTIE_DISPATCH(dtype, X, (token_shift_kernel<8, X><<<grid, threads, 0, stream>>>(
        static_cast<const X*>(x), mu, mixes, state, static_cast<X*>(out), cu_q, token_request, state_slots, C, T)));
  } else {
    DISTIE_DISPATCH(dtype, X, (token_shift_kernel<1, X><<<grid, threads, 0, stream>>>(
        static_cast<const X*>(x), mu, mixes, state, static_cast<X*>(out), cu_q, token_request, state_slots, C, T)));
  }
  return launch_status();
}

extern "C" int distie_wkv_scan_max_dim() { return 256; }
extern "C" int distie_wkv_scan_max_rank() { return 8192; }

// r, k, v, gates: [T, H * D] of `dtype` with rows `ld` apart; low: [T, rank] of `low_dtype`, rows `ld_low` apart
extern "C" int distie_wkv_scan(const void* r, const void* k, const void* v, const void* gates, int dtype, int64_t ld,
                               const void* low, int low_dtype, int64_t ld_low, int rank, const float* up,
                               const float* up_bias, const float* bonus, float* state, const float* norm_weight, float eps,
                               void* out, int out_dtype, const int32_t* cu_q, const int32_t* state_slots, int B, int H,
                               int D, hipStream_t stream) {
  if (B <= 0) return 0;
  if (H < 1 || D < 1 || D > 256 || rank < 1 || rank > 8192 || ld < static_cast<int64_t>(H) * D || ld_low < rank || !(eps >= 0.f))
    return DISTIE_BAD_ARGUMENT;
  const dim3 grid(B, H);
  const size_t lds = static_cast<size_t>(rank) * sizeof(float);
#define DISTIE_WKV_SCAN(COLS, PARTS, ROWS)                                                                               \
  DISTIE_DISPATCH(dtype, X, DISTIE_DISPATCH(low_dtype, L, DISTIE_DISPATCH(out_dtype, O, (                                \
      wkv_scan_kernel<X, L, O, COLS, PARTS, ROWS><<<grid, COLS * PARTS, lds, stream>>>(                                  \
          static_cast<const X*>(r), static_cast<const X*>(k), static_cast<const X*>(v), static_cast<const X*>(gates),    \
          ld, static_cast<const L*>(low), ld_low, rank, up, up_bias, bonus, state, norm_weight, eps,                     \
          static_cast<O*>(out), cu_q, state_slots, H, D)))))
  if (D <= 32) {
    DISTIE_WKV_SCAN(64, 4, 8);
  } else if (D <= 64) {
    DISTIE_WKV_SCAN(64, 4, 16);
  } else if (D <= 128) {
    DISTIE_WKV_SCAN(128, 4, 32);
  } else {
    DISTIE_WKV_SCAN(256, 4, 64);
  }
#undef DISTIE_WKV_SCAN
  return launch_status();
}

extern "C" int distie_wkv_chunk_rows() { return WK_ROWS; }
extern "C" int distie_wkv_chunked_max_dim() { return 128; }

// z: float32 [T, H * D]; chunks: int32 [num_chunks][4] = {request, first row, rows (1..64), 0}, the chunks of a request one
// after the other; request_chunks: int32 [B + 1]; scratch: float32 [num_chunks, H, D, D]; totals: float32 [num_chunks, H, D]
extern "C" int distie_wkv_scan_chunked(const void* r, const void* k, const void* v, const void* gates, int dtype, int64_t ld,
                                       const float* z, const float* bonus, float* state, const float* norm_weight, float eps,
                                       void* out, int out_dtype, float* scratch, float* totals, const int32_t* chunks,
                                       const int32_t* request_chunks, const int32_t* state_slots, int num_chunks, int B,
                                       int H, int D, hipStream_t stream) {
  if (B <= 0 || num_chunks <= 0) return 0;
  if (H < 1 || D < 1 || D > 128 || ld < static_cast<int64_t>(H) * D || !(eps >= 0.f)) return DISTIE_BAD_ARGUMENT;
  const int4* table = reinterpret_cast<const int4*>(chunks);
  const dim3 grid(num_chunks, H);
  const auto aligned = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  const int vectors = ld % 4 == 0 && aligned(r) && aligned(k) && aligned(v) && aligned(z) && aligned(scratch) ? 1 : 0;
  int status = 0;
#define DISTIE_WKV_CHUNKS(DP)                                                                                            \
  DISTIE_DISPATCH(dtype, X, DISTIE_DISPATCH(out_dtype, O, {                                                              \
    constexpr int LDS = (WK_ROWS * (DP + 4) + DP * DP + WK_ROWS * DP + 4 * DP) * static_cast<int>(sizeof(float));        \
    const int whole = vectors && D == DP ? 1 : 0;                                                                        \
    if (LDS > 48 * 1024 &&                                                                                               \
        hipFuncSetAttribute(reinterpret_cast<const void*>(wkv_chunk_outputs_kernel<DP, X, O>),                           \
                            hipFuncAttributeMaxDynamicSharedMemorySize, LDS) != hipSuccess)                              \
      return DISTIE_BAD_ARGUMENT;                                                                                        \
    wkv_chunk_sums_kernel<DP, X><<<grid, 256, 0, stream>>>(static_cast<const X*>(k), static_cast<const X*>(v), ld, z,    \
                                                           scratch, totals, table, H, D, whole);                         \
    if ((status = launch_status()) != 0) return status;                                                                  \
    wkv_chunk_states_kernel<<<dim3(B, H, (D * D + 255) / 256), 256, 0, stream>>>(scratch, totals, state, request_chunks, \
                                                                                state_slots, H, D);                      \
    if ((status = launch_status()) != 0) return status;                                                                  \
    wkv_chunk_outputs_kernel<DP, X, O><<<grid, 256, LDS, stream>>>(                                                      \
        static_cast<const X*>(r), static_cast<const X*>(k), static_cast<const X*>(v), static_cast<const X*>(gates), ld,  \
        z, bonus, scratch, norm_weight, eps, static_cast<O*>(out), table, H, D, whole);                                  \
  }))
  if (D <= 16) {
    DISTIE_WKV_CHUNKS(16);
  } else if (D <= 32) {
    DISTIE_WKV_CHUNKS(32);
  } else if (D <= 48) {
    DISTIE_WKV_CHUNKS(48);
  } else if (D <= 64) {
    DISTIE_WKV_CHUNKS(64);
  } else if (D <= 96) {
    DISTIE_WKV_CHUNKS(96);
  } else {
    DISTIE_WKV_CHUNKS(128);
  }
#undef DISTIE_WKV_CHUNKS
  return launch_status();
}

// tanh of a [T, N] float32 view (rows `ld` apart) into a dense tensor
extern "C" int distie_tanh_f32(const float* in, int64_t ld, float* out, int T, int N, hipStream_t stream) {
  if (T <= 0) return 0;
  if (N < 1 || ld < N) return DISTIE_BAD_ARGUMENT;
  const int64_t blocks = (static_cast<int64_t>(T) * N + 255) / 256;
  if (blocks > 0x7fffffff) return DISTIE_BAD_ARGUMENT;
  tanh_f32_kernel<<<static_cast<unsigned>(blocks), 256, 0, stream>>>(in, ld, out, N, T);
  return launch_status();
}
