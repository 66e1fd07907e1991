// The gated delta rule: a state per head that forgets by a factor computed from the token and corrects what it holds under
// the token's key.
//
// qkv [T, ld] holds q (G heads of D), k (G heads of D), v (H heads of E); head h reads q/k head h / (H / G). b and a: one
// logit a head and row. With q^ = q / sqrt(sum(q^2) + unit_eps) * q_scale, k^ = k / sqrt(sum(k^2) + unit_eps),
// w = sigmoid(b), ln f = -exp(a_log) * softplus(a + dt_bias), per head
//     S <- f S (D x E, float32),   u = w (v - S^T k^),   S <- S + k^ u^T,   o = S^T q^.
// state float32 [slots, H, D, E]. Unit norms, w, f, the state and every sum are float32 in either precision.
//
// A step is a flattened batch: request b's new tokens are rows cu_q[b] .. cu_q[b+1]-1, its state row state_slots[b].
#include "common.h"

namespace {

__device__ __forceinline__ float sigmoidf(float x) { return 1.f / (1.f + expf(-x)); }
__device__ __forceinline__ float softplusf(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

// ---------------------------------------------------------------------------------------------------
// Row after row. A block owns 64 columns e of one head of one request; wave `part` keeps the state's rows d = part * ROWS
// .. + ROWS - 1 of its lanes' columns in registers. Every wave fetches all of q and k (lane: dimensions lane, lane + 64,
// ...), so it has the sums of their squares and their product without a barrier, and keeps them in rows of LDS of its own.
// With S the state in front of the row: S^T k^ and S^T q^ are summed in one walk, their parts meet in LDS (two sets of
// places in turn: one barrier a row), and o = f S^T q^ + (k^ . q^) u. The next row's inputs are asked for before this row's
// are used.
template <typename X, int PARTS, int ROWS>
__global__ void __launch_bounds__(64 * PARTS)
delta_scan_kernel(const X* __restrict__ qkv, int64_t ld, const X* __restrict__ beta, int64_t ldb, const X* __restrict__ decay,
                  int64_t lda, const float* __restrict__ a_log, const float* __restrict__ dt_bias, float* __restrict__ state,
                  float* __restrict__ out, const int32_t* __restrict__ cu_q, const int32_t* __restrict__ state_slots, int H,
                  int G, int D, int E, float q_scale, float unit_eps) {
  constexpr int PER = PARTS * ROWS / 64;                 // dimensions of q and k a lane fetches
  __shared__ float q_s[PARTS][PARTS * ROWS], k_s[PARTS][PARTS * ROWS];
  __shared__ float partial[2][PARTS][2][64];
  const int b = blockIdx.x, head = blockIdx.y;
  const int lane = threadIdx.x % 64, part = threadIdx.x / 64;
  const int e = blockIdx.z * 64 + lane;
  const int first = cu_q[b], last = cu_q[b + 1];
  if (first >= last) return;
  const int shared_head = head / (H / G);
  const float rate = -expf(a_log[head]), bias = dt_bias[head];
  const int64_t q_at = static_cast<int64_t>(shared_head) * D, k_at = static_cast<int64_t>(G + shared_head) * D;
  const int64_t v_at = 2 * static_cast<int64_t>(G) * D + static_cast<int64_t>(head) * E + e;
  float* own = state + (static_cast<int64_t>(state_slots[b]) * H + head) * D * E;
  const int d0 = part * ROWS;
  float s[ROWS];
#pragma unroll
  for (int r = 0; r < ROWS; ++r) s[r] = (d0 + r < D && e < E) ? own[static_cast<int64_t>(d0 + r) * E + e] : 0.f;
  float nq[PER], nk[PER], nv = 0.f, nb = 0.f, na = 0.f;
  auto fetch = [&](int t) {
    const X* row = qkv + static_cast<int64_t>(t) * ld;
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int d = lane + 64 * i;
      nq[i] = d < D ? to_float(row[q_at + d]) : 0.f;
      nk[i] = d < D ? to_float(row[k_at + d]) : 0.f;
    }
    nv = e < E ? to_float(row[v_at]) : 0.f;
    nb = to_float(beta[static_cast<int64_t>(t) * ldb + head]);
    na = to_float(decay[static_cast<int64_t>(t) * lda + head]);
  };
  fetch(first);
  for (int t = first; t < last; ++t) {
    float qq = 0.f, kk = 0.f, qk = 0.f;
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      q_s[part][lane + 64 * i] = nq[i];
      k_s[part][lane + 64 * i] = nk[i];
      qq += nq[i] * nq[i];
      kk += nk[i] * nk[i];
      qk += nq[i] * nk[i];
    }
    __builtin_amdgcn_wave_barrier();
    const float v = nv, w = sigmoidf(nb), f = expf(rate * softplusf(na + bias));
    if (t + 1 < last) fetch(t + 1);
    const float q_unit = q_scale / sqrtf(wave_sum(qq) + unit_eps), k_unit = 1.f / sqrtf(wave_sum(kk) + unit_eps);
    const float both = wave_sum(qk) * q_unit * k_unit;
    float by_k = 0.f, by_q = 0.f;
#pragma unroll
    for (int r = 0; r < ROWS; ++r) {
      by_k += s[r] * k_s[part][d0 + r];
      by_q += s[r] * q_s[part][d0 + r];
    }
    float(*place)[2][64] = partial[t & 1];
    place[part][0][lane] = by_k;
    place[part][1][lane] = by_q;
    __syncthreads();
    float all_k = 0.f, all_q = 0.f;
#pragma unroll
    for (int p = 0; p < PARTS; ++p) all_k += place[p][0][lane], all_q += place[p][1][lane];
    const float u = w * (v - f * (all_k * k_unit));
    const float ku = k_unit * u;
#pragma unroll
    for (int r = 0; r < ROWS; ++r) s[r] = f * s[r] + k_s[part][d0 + r] * ku;
    if (part == 0 && e < E) out[(static_cast<int64_t>(t) * H + head) * E + e] = f * (all_q * q_unit) + both * u;
  }
#pragma unroll
  for (int r = 0; r < ROWS; ++r)
    if (d0 + r < D && e < E) own[static_cast<int64_t>(d0 + r) * E + e] = s[r];
}

// ---------------------------------------------------------------------------------------------------
// Portions of prompts, in chunks of L = 64 rows. With l_i the running sum of ln f inside the chunk (falling, <= 0) and S
// the state in front of it, the chunk's corrections u solve a triangular system,
//     u_i + sum_{j<i} A_ij u_j = w_i (v_i - exp(l_i) S^T k^_i),      A_ij = w_i exp(l_i - l_j) (k^_i . k^_j),
// so with X the solution of (I + A) X = (w_i exp(l_i) k^_i | w_i v_i), X = (W | V'):     U = V' - W S,
//     S_next = exp(l_L) S + sum_j exp(l_L - l_j) k^_j u_j^T,
//     o_i    = exp(l_i) S^T q^_i + sum_{j<=i} exp(l_i - l_j) (q^_i . k^_j) u_j.
// Every exponent is <= 0 and no quotient of decays is formed.
//   prepare (chunk, head side by side): W, V', the factors k~_j = exp(l_L - l_j) k^_j (transposed), the pairs' weights in o
//   states  (request, head, 16 columns e): U and the state in front of every chunk, chunk after chunk
//   outputs (chunk, head, 64 columns): o
// Float32 throughout, products on float32 matrix products. Scratch is padded: DP = D rounded up to a multiple of 64 that
// four waves share evenly (64, 128 or 256), EP = E rounded up to a multiple of 16, zeros beyond D, E and a chunk's rows. It
// lies in tiles of 16 x 16 in the order in which a wave of `states` holds them, lane (g = lane / 16, c = lane % 16) four
// neighbouring values, so that the wave reads and writes a tile as one run of 1,024 bytes:
//   W       [chunk, head][rows / 16][DP / 16]:    lane holds row c, columns 4 g ..
//   k~      [chunk, head][DP / 16][rows / 16]:    lane holds dimension c, rows 4 g ..
//   V', U   [chunk, head][EP / 16][rows / 16]:    lane holds rows 4 g .., column c
//   states  [chunk, head][EP / 16][DP / 16]:      lane holds dimensions 4 g .., column c
// A chunk's table entry is {request, first row, rows, unused}.
constexpr int DL = 64;
constexpr int DL_PAD = DL + 1;
constexpr int DL_ROW = DL + 4;          // row stride of the triangular matrix: 16-byte reads of a row
typedef __attribute__((__vector_size__(16 * sizeof(float)))) float delta_floatx16;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float delta_floatx4;
__device__ __forceinline__ int tile_row(int v, int lane) { return 8 * (v / 4) + 4 * (lane / 32) + v % 4; }

// a[k] of thread q of four neighbours <-> a[q] of thread k
__device__ __forceinline__ void transpose_quad(float a[4]) {
  const int q = threadIdx.x % 4;
  const auto swap = [](float& low, float& high, bool upper, float partner) {
    if (upper) low = partner;
    else high = partner;
  };
  const auto near = [](float x) { return __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(x), 0xB1, 0xf, 0xf, true)); };
  const auto far = [](float x) { return __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(x), 0x4E, 0xf, 0xf, true)); };
  const bool odd = q & 1, upper = q & 2;
  swap(a[0], a[1], odd, near(odd ? a[0] : a[1]));
  swap(a[2], a[3], odd, near(odd ? a[2] : a[3]));
  swap(a[0], a[2], upper, far(upper ? a[0] : a[2]));
  swap(a[1], a[3], upper, far(upper ? a[1] : a[3]));
}

template <typename X>
__global__ void __launch_bounds__(256, 2)
delta_chunk_prepare_kernel(const X* __restrict__ qkv, int64_t ld, const X* __restrict__ beta, int64_t ldb,
                           const X* __restrict__ decay, int64_t lda, const float* __restrict__ a_log,
                           const float* __restrict__ dt_bias, float* __restrict__ w_out, float* __restrict__ v_out,
                           float* __restrict__ k_out, float* __restrict__ pairs, float* __restrict__ q_factor,
                           float* __restrict__ totals, const int4* __restrict__ chunks, int H, int G, int D, int E, int DP,
                           int EP, float q_scale, float unit_eps) {
  __shared__ float l_s[DL], beta_s[DL], q_unit[DL], k_unit[DL];
  __shared__ float in_factor[DL], out_factor[DL];        // w_i exp(l_i) and exp(l_L - l_i), each over the length of k_i
  __shared__ float q_s[DL][DL_PAD], k_s[DL][DL_PAD];     // [row][d of this pass]
  __shared__ __attribute__((aligned(16))) float a_s[DL][DL_ROW];
  const int chunk = blockIdx.x, head = blockIdx.y;
  const int4 entry = chunks[chunk];
  const int first = entry.y, rows = entry.z;
  const int shared_head = head / (H / G);
  const int tid = threadIdx.x, lane = tid % 64, wave = tid / 64;
  const int64_t q_at = static_cast<int64_t>(shared_head) * D, k_at = static_cast<int64_t>(G + shared_head) * D;
  const int64_t place = static_cast<int64_t>(chunk) * H + head;
  if (wave == 0) {
    const bool in = lane < rows;
    const int64_t t = first + min(lane, rows - 1);
    float l = in ? -expf(a_log[head]) * softplusf(to_float(decay[t * lda + head]) + dt_bias[head]) : 0.f;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float before = __shfl_up(l, o, 64);
      if (lane >= o) l += before;
    }
    l_s[lane] = l;
    beta_s[lane] = in ? sigmoidf(to_float(beta[t * ldb + head])) : 0.f;
  }
  // k . k and q . k of the chunk's rows (a wave: 32 rows i by 32 rows j), and the sums of squares (four threads a row)
  const int ib = 32 * (wave / 2), jb = 32 * (wave % 2);
  const int sum_row = tid / 4, sum_part = tid % 4;
  delta_floatx16 kk = {}, qk = {};
  float q_sq = 0.f, k_sq = 0.f;
  for (int n0 = 0; n0 < D; n0 += DL) {
    __syncthreads();
    {
      // a tile's loads are under way together: addresses clamped into the step's rows, what does not belong is dropped
      const X* from = qkv + static_cast<int64_t>(first) * ld + min(n0 + lane, D - 1);
      X q[16], k[16];
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int64_t at = static_cast<int64_t>(min(wave + 4 * r, rows - 1)) * ld;
        q[r] = from[at + q_at];
        k[r] = from[at + k_at];
      }
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int j = wave + 4 * r;
        const bool in = j < rows && n0 + lane < D;
        q_s[j][lane] = in ? to_float(q[r]) : 0.f;
        k_s[j][lane] = in ? to_float(k[r]) : 0.f;
      }
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const float q = q_s[sum_row][4 * i + sum_part], k = k_s[sum_row][4 * i + sum_part];
      q_sq += q * q;
      k_sq += k * k;
    }
    if (jb <= ib) {
      for (int n = 0; n < DL; n += 2) {
        const float other = k_s[jb + lane % 32][n + lane / 32];
        kk = __builtin_amdgcn_mfma_f32_32x32x2f32(k_s[ib + lane % 32][n + lane / 32], other, kk, 0, 0, 0);
        qk = __builtin_amdgcn_mfma_f32_32x32x2f32(q_s[ib + lane % 32][n + lane / 32], other, qk, 0, 0, 0);
      }
    }
  }
  q_sq += __shfl_xor(q_sq, 1, 64);
  k_sq += __shfl_xor(k_sq, 1, 64);
  q_sq += __shfl_xor(q_sq, 2, 64);
  k_sq += __shfl_xor(k_sq, 2, 64);
  if (sum_part == 0) {
    q_unit[sum_row] = q_scale / sqrtf(q_sq + unit_eps);
    k_unit[sum_row] = 1.f / sqrtf(k_sq + unit_eps);
  }
  __syncthreads();
  const float l_end = l_s[DL - 1];                       // (rows beyond the chunk add nothing)
  float* pair = pairs + place * DL * DL;
#pragma unroll
  for (int v = 0; v < 16; ++v) {
    const int i = ib + tile_row(v, lane), j = jb + lane % 32;
    const float fade = j <= i && i < rows ? expf(l_s[i] - l_s[j]) * k_unit[j] : 0.f;
    a_s[i][j] = j < i ? fade * beta_s[i] * k_unit[i] * kk[v] : 0.f;
    pair[i * DL + j] = fade * q_unit[i] * qk[v];
  }
  if (tid < DL) {
    const float l = expf(l_s[tid]);
    q_factor[place * DL + tid] = l * q_unit[tid];
    in_factor[tid] = beta_s[tid] * k_unit[tid] * l;
    out_factor[tid] = k_unit[tid] * expf(l_end - l_s[tid]);
  }
  if (tid == 0) totals[place] = expf(l_end);
  __syncthreads();
  // (I + A) X = B, a thread a column of B, forward substitution with the column in registers
  for (int c = tid; c < DP + EP; c += 256) {
    const bool key = c < DP;
    const int col = key ? c : c - DP;
    const bool in = key ? col < D : col < E;
    const X* from = qkv + static_cast<int64_t>(first) * ld +
                    (key ? k_at + col : 2 * static_cast<int64_t>(G) * D + static_cast<int64_t>(head) * E + col);
    float x[DL];
#pragma unroll
    for (int i = 0; i < DL; ++i) x[i] = to_float(from[in ? min(i, rows - 1) * ld : 0]);      // (every load under way together)
    if (!in) {
#pragma unroll
      for (int i = 0; i < DL; ++i) x[i] = 0.f;
    }
    if (key) {
      float* to = k_out + (place * DP + col / 16 * 16) * DL + col % 16 * 4;
#pragma unroll
      for (int i = 0; i < DL; i += 4) {
        float4 k4;
        k4.x = i < rows ? x[i] * out_factor[i] : 0.f;
        k4.y = i + 1 < rows ? x[i + 1] * out_factor[i + 1] : 0.f;
        k4.z = i + 2 < rows ? x[i + 2] * out_factor[i + 2] : 0.f;
        k4.w = i + 3 < rows ? x[i + 3] * out_factor[i + 3] : 0.f;
        *reinterpret_cast<float4*>(to + i / 16 * 256 + i / 4 % 4 * 64) = k4;
      }
    }
#pragma unroll
    for (int i = 0; i < DL; ++i) {
      // (rows beyond the chunk have no factor; four sums, so that a sum need not wait for the one before)
      float acc = x[i] * (key ? in_factor[i] : beta_s[i]), more[3] = {};
#pragma unroll
      for (int j = 0; j < i; j += 4) {
        const float4 a = *reinterpret_cast<const float4*>(&a_s[i][j]);       // (zero from the diagonal on)
        acc -= a.x * x[j];
        if (j + 1 < i) more[0] -= a.y * x[j + 1];
        if (j + 2 < i) more[1] -= a.z * x[j + 2];
        if (j + 3 < i) more[2] -= a.w * x[j + 3];
      }
      acc += more[0] + (more[1] + more[2]);
      x[i] = acc;
    }
    if (key) {
      // four neighbouring columns change places with four rows: a thread then holds one row's four columns
      float* to = w_out + place * DL * DP + col / 16 * 256 + col / 4 % 4 * 64 + tid % 4 * 4;
#pragma unroll
      for (int i = 0; i < DL; i += 4) {
        transpose_quad(x + i);
        *reinterpret_cast<float4*>(to + i / 16 * (DP / 16) * 256 + i % 16 * 4) = float4{x[i], x[i + 1], x[i + 2], x[i + 3]};
      }
    } else {
      float* to = v_out + (place * EP + col / 16 * 16) * DL + col % 16 * 4;
#pragma unroll
      for (int i = 0; i < DL; i += 4)
        *reinterpret_cast<float4*>(to + i / 16 * 256 + i / 4 % 4 * 64) = float4{x[i], x[i + 1], x[i + 2], x[i + 3]};
    }
  }
}

// blockIdx = (request, head, 16 columns e). Wave w keeps rows d = 16 TILES w .. of the state's 16 columns as TILES tiles of
// 16 x 16 in the products' own result layout: lane (g = lane / 16, c = lane % 16) holds rows 4 g + v and column c of a tile,
// which is also what the second operand of v_mfma_f32_16x16x4_f32 takes if the four products of a step of 16 summed indexes
// take index 4 g + t from lane group g at product t. So neither the state nor U moves between lanes; W and k~ lie in that
// order too. The four waves' shares of W S meet in LDS (two sets of places in turn: one barrier a chunk),
// and every wave adds them up for itself.
template <int TILES>
__global__ void __launch_bounds__(256, 1)
delta_chunk_states_kernel(const float* __restrict__ w_in, const float* __restrict__ v_in, const float* __restrict__ k_in,
                          const float* __restrict__ totals, float* __restrict__ u_out, float* __restrict__ scratch,
                          float* __restrict__ state, const int32_t* __restrict__ first_chunk,
                          const int32_t* __restrict__ state_slots, int H, int D, int E, int EP) {
  constexpr int DP = 64 * TILES;
  __shared__ __attribute__((aligned(16))) float share[2][4][4][64 * 4];        // [turn][wave][tile of rows][lane, v]
  const int b = blockIdx.x, head = blockIdx.y, e0 = blockIdx.z * 16;
  const int begin = first_chunk[b], end = first_chunk[b + 1];
  if (begin >= end) return;
  const int lane = threadIdx.x % 64, wave = threadIdx.x / 64;
  const int g = lane / 16, c = lane % 16;
  const int d0 = 16 * TILES * wave;
  const bool column = e0 + c < E;
  float* own = state + (static_cast<int64_t>(state_slots[b]) * H + head) * D * E + e0 + c;
  delta_floatx4 s[TILES];
#pragma unroll
  for (int i = 0; i < TILES; ++i)
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const int d = d0 + 16 * i + 4 * g + v;
      s[i][v] = column && d < D ? own[static_cast<int64_t>(d) * E] : 0.f;
    }
  // What a chunk needs is asked for while the chunk in front of it is worked on, into the other of two sets of registers
  // (wider states have registers for one set only: asked for as soon as the set is free).
  constexpr int SETS = TILES <= 2 ? 2 : 1;
  delta_floatx4 w4[SETS][4][TILES], k4[SETS][TILES][4];
  delta_floatx4 v4[SETS][4];
  float total_of[SETS];
  auto fetch_w = [&](int set, int chunk) {
    const int64_t place = static_cast<int64_t>(min(chunk, end - 1)) * H + head;
    const float* p = w_in + place * DL * DP + TILES * wave * 256 + 4 * lane;
#pragma unroll
    for (int m = 0; m < 4; ++m)
#pragma unroll
      for (int i = 0; i < TILES; ++i) w4[set][m][i] = *reinterpret_cast<const delta_floatx4*>(p + (m * (DP / 16) + i) * 256);
  };
  auto fetch_kv = [&](int set, int chunk) {
    const int64_t place = static_cast<int64_t>(min(chunk, end - 1)) * H + head;
    const float* q = v_in + (place * EP + e0) * DL + 4 * lane;
#pragma unroll
    for (int m = 0; m < 4; ++m) v4[set][m] = *reinterpret_cast<const delta_floatx4*>(q + m * 256);
    total_of[set] = totals[place];
    const float* p = k_in + (place * DP + d0) * DL + 4 * lane;
#pragma unroll
    for (int i = 0; i < TILES; ++i)
#pragma unroll
      for (int m = 0; m < 4; ++m) k4[set][i][m] = *reinterpret_cast<const delta_floatx4*>(p + (4 * i + m) * 256);
  };
  delta_floatx4 mine = {};                                 // the rows of U that this wave hands on: tile `wave`
  auto store_u = [&](int chunk) {
    *reinterpret_cast<delta_floatx4*>(u_out + ((static_cast<int64_t>(chunk) * H + head) * EP + e0) * DL + wave * 256 + 4 * lane) = mine;
  };
  auto work = [&](int chunk, int set) {
    const int64_t place = static_cast<int64_t>(chunk) * H + head;
    // stores first, so that they are a chunk old when the next wait for loads comes: the state in front of the chunk, and the
    // chunk before's U
    float* to = scratch + (place * EP + e0) * DP + TILES * wave * 256 + 4 * lane;
#pragma unroll
    for (int i = 0; i < TILES; ++i) *reinterpret_cast<delta_floatx4*>(to + i * 256) = s[i];
    if (chunk > begin) store_u(chunk - 1);
    if constexpr (SETS == 2) {
      fetch_w(1 - set, chunk + 1);
      fetch_kv(1 - set, chunk + 1);
      __builtin_amdgcn_sched_barrier(0);
    }
    delta_floatx4 part[4] = {};
#pragma unroll
    for (int i = 0; i < TILES; ++i)
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int m = 0; m < 4; ++m) part[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(w4[set][m][i][t], s[i][t], part[m], 0, 0, 0);
    if constexpr (SETS == 1) fetch_w(0, chunk + 1);
    float(*at)[4][256] = share[(chunk - begin) & 1];
#pragma unroll
    for (int m = 0; m < 4; ++m) *reinterpret_cast<delta_floatx4*>(&at[wave][m][4 * lane]) = part[m];
    __syncthreads();
    float u[4][4];
#pragma unroll
    for (int m = 0; m < 4; ++m) {
      delta_floatx4 sum = *reinterpret_cast<const delta_floatx4*>(&at[0][m][4 * lane]);
#pragma unroll
      for (int w = 1; w < 4; ++w) {
        const delta_floatx4 more = *reinterpret_cast<const delta_floatx4*>(&at[w][m][4 * lane]);
#pragma unroll
        for (int v = 0; v < 4; ++v) sum[v] += more[v];
      }
#pragma unroll
      for (int v = 0; v < 4; ++v) u[m][v] = v4[set][m][v] - sum[v];
    }
#pragma unroll
    for (int m = 0; m < 4; ++m)
#pragma unroll
      for (int v = 0; v < 4; ++v) mine[v] = m == wave ? u[m][v] : mine[v];
#pragma unroll
    for (int i = 0; i < TILES; ++i)
#pragma unroll
      for (int v = 0; v < 4; ++v) s[i][v] *= total_of[set];
#pragma unroll
    for (int m = 0; m < 4; ++m)
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int i = 0; i < TILES; ++i) s[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(k4[set][i][m][t], u[m][t], s[i], 0, 0, 0);
    if constexpr (SETS == 1) fetch_kv(0, chunk + 1);
  };
  fetch_w(0, begin);
  fetch_kv(0, begin);
  for (int chunk = begin; chunk < end; chunk += SETS) {
    work(chunk, 0);
    if constexpr (SETS == 2) {
      if (chunk + 1 < end) work(chunk + 1, 1);
    }
  }
  store_u(end - 1);
  if (column) {
#pragma unroll
    for (int i = 0; i < TILES; ++i)
#pragma unroll
      for (int v = 0; v < 4; ++v) {
        const int d = d0 + 16 * i + 4 * g + v;
        if (d < D) own[static_cast<int64_t>(d) * E] = s[i][v];
      }
  }
}

// blockIdx = (chunk, head, 64 columns e); a wave: 32 rows i by 32 columns
template <typename X>
__global__ void __launch_bounds__(256)
delta_chunk_outputs_kernel(const X* __restrict__ qkv, int64_t ld, const float* __restrict__ q_factor,
                           const float* __restrict__ pairs, const float* __restrict__ u_in, const float* __restrict__ scratch,
                           float* __restrict__ out, const int4* __restrict__ chunks, int H, int G, int D, int E, int DP,
                           int EP) {
  __shared__ float a_s[DL][DL_PAD];     // a tile of q [i][d], then the pairs' weights [i][j]
  __shared__ float b_s[DL][DL_PAD];     // a tile of the state [d][e], then U [j][e]
  __shared__ float f_s[DL];
  const int chunk = blockIdx.x, head = blockIdx.y, e0 = blockIdx.z * 64;
  const int4 entry = chunks[chunk];
  const int first = entry.y, rows = entry.z;
  const int lane = threadIdx.x % 64, wave = threadIdx.x / 64;
  const int64_t place = static_cast<int64_t>(chunk) * H + head;
  const int64_t q_at = static_cast<int64_t>(head / (H / G)) * D;
  if (threadIdx.x < DL) f_s[threadIdx.x] = q_factor[place * DL + threadIdx.x];
  const int ib = 32 * (wave / 2), pb = 32 * (wave % 2);
  const float* s_in = scratch + place * DP * EP;
  // four tiles of the wave's 16 columns -> rows of b_s
  auto spread = [&](const float4 tiles[4]) {
#pragma unroll
    for (int m = 0; m < 4; ++m) {
      const int row = 16 * m + 4 * (lane / 16), col = 16 * wave + lane % 16;
      b_s[row][col] = tiles[m].x;
      b_s[row + 1][col] = tiles[m].y;
      b_s[row + 2][col] = tiles[m].z;
      b_s[row + 3][col] = tiles[m].w;
    }
  };
  delta_floatx16 y = {};
  for (int n0 = 0; n0 < D; n0 += DL) {
    __syncthreads();
    const X* q_from = qkv + static_cast<int64_t>(first) * ld + q_at + min(n0 + lane, D - 1);
    X q[16];
    float4 s[4];
#pragma unroll
    for (int r = 0; r < 16; ++r) q[r] = q_from[static_cast<int64_t>(min(wave + 4 * r, rows - 1)) * ld];
    // a wave: the 16 columns 16 wave .., four tiles of 16 dimensions (zeros beyond D, up to DP)
    const float* s_from = s_in + static_cast<int64_t>(min(e0 + 16 * wave, EP - 16)) * DP + n0 / 16 * 256 + 4 * lane;
#pragma unroll
    for (int m = 0; m < 4; ++m) s[m] = *reinterpret_cast<const float4*>(s_from + m * 256);
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int j = wave + 4 * r;
      a_s[j][lane] = j < rows && n0 + lane < D ? to_float(q[r]) : 0.f;
    }
    spread(s);
    __syncthreads();
    for (int n = 0; n < DL; n += 2)
      y = __builtin_amdgcn_mfma_f32_32x32x2f32(a_s[ib + lane % 32][n + lane / 32], b_s[n + lane / 32][pb + lane % 32], y, 0, 0, 0);
  }
#pragma unroll
  for (int v = 0; v < 16; ++v) y[v] *= f_s[ib + tile_row(v, lane)];
  float p[16];
  float4 u[4];
#pragma unroll
  for (int r = 0; r < 16; ++r) p[r] = pairs[place * DL * DL + (wave + 4 * r) * DL + lane];
  const float* u_from = u_in + (place * EP + min(e0 + 16 * wave, EP - 16)) * DL + 4 * lane;
#pragma unroll
  for (int m = 0; m < 4; ++m) u[m] = *reinterpret_cast<const float4*>(u_from + m * 256);
  __syncthreads();
#pragma unroll
  for (int r = 0; r < 16; ++r) a_s[wave + 4 * r][lane] = p[r];
  spread(u);
  __syncthreads();
  for (int j = 0; j < ib + 32; j += 2)
    y = __builtin_amdgcn_mfma_f32_32x32x2f32(a_s[ib + lane % 32][j + lane / 32], b_s[j + lane / 32][pb + lane % 32], y, 0, 0, 0);
#pragma unroll
  for (int v = 0; v < 16; ++v) {
    const int i = ib + tile_row(v, lane), col = e0 + pb + lane % 32;
    if (i < rows && col < E) out[(static_cast<int64_t>(first + i) * H + head) * E + col] = y[v];
  }
}

bool bad_shape(int H, int G, int D, int E, int64_t ld, int64_t ldb, int64_t lda) {
  return H < 1 || G < 1 || H % G != 0 || D < 1 || E < 1 || D > 256 || H > 65535 || ldb < H || lda < H ||
         ld < 2 * static_cast<int64_t>(G) * D + static_cast<int64_t>(H) * E;
}

}  // namespace

// the largest key size a head may have
extern "C" int distie_delta_scan_max_dim() { return 256; }

extern "C" int distie_delta_scan(const void* qkv, int dtype, int64_t ld, const void* beta, int64_t ldb, const void* decay,
                                 int64_t lda, const float* a_log, const float* dt_bias, float* state, float* out,
                                 const int32_t* cu_q, const int32_t* state_slots, int B, int H, int G, int D, int E,
                                 float q_scale, float unit_eps, hipStream_t stream) {
  if (B <= 0) return 0;
  if (bad_shape(H, G, D, E, ld, ldb, lda)) return DISTIE_BAD_ARGUMENT;
  const dim3 grid(B, H, (E + 63) / 64);
#define DISTIE_DELTA(PARTS, ROWS)                                                                                     \
  DISTIE_DISPATCH(dtype, X, (delta_scan_kernel<X, PARTS, ROWS><<<grid, 64 * PARTS, 0, stream>>>(                      \
      static_cast<const X*>(qkv), ld, static_cast<const X*>(beta), ldb, static_cast<const X*>(decay), lda, a_log,     \
      dt_bias, state, out, cu_q, state_slots, H, G, D, E, q_scale, unit_eps)))
  if (D <= 64) {
    DISTIE_DELTA(4, 16);
  } else if (D <= 128) {
    DISTIE_DELTA(4, 32);
  } else {
    DISTIE_DELTA(8, 32);
  }
#undef DISTIE_DELTA
  return launch_status();
}

extern "C" int distie_delta_scan_chunk_rows() { return DL; }
extern "C" int distie_delta_scan_padded_dim(int D) { return D <= 64 ? 64 : (D <= 128 ? 128 : 256); }

// chunks: int32 [count][4] = {request, first row, rows (1..64), 0}, the chunks of a request one after the other;
// first_chunk: int32 [B + 1]. Float32 scratch, DP = distie_delta_scan_padded_dim(D), EP = E rounded up to a multiple of 16
// (numbers of elements; for their order see above): w [count, H, 64, DP], v and u [count, H, 64, EP], k [count, H, DP, 64], pairs [count, H, 64, 64], q_factor [count, H, 64],
// totals [count, H], states [count, H, DP, EP].
extern "C" int distie_delta_scan_chunked(const void* qkv, int dtype, int64_t ld, const void* beta, int64_t ldb,
                                         const void* decay, int64_t lda, const float* a_log, const float* dt_bias,
                                         float* state, float* out, float* w, float* v, float* u, float* k, float* pairs,
                                         float* q_factor, float* totals, float* states, const void* chunks,
                                         const int32_t* first_chunk, const int32_t* state_slots, int count, int B, int H,
                                         int G, int D, int E, float q_scale, float unit_eps, hipStream_t stream) {
  if (B <= 0 || count <= 0) return 0;
  if (bad_shape(H, G, D, E, ld, ldb, lda)) return DISTIE_BAD_ARGUMENT;
  const int DP = distie_delta_scan_padded_dim(D), EP = (E + 15) / 16 * 16;
  const int4* table = static_cast<const int4*>(chunks);
  int status = 0;
  DISTIE_DISPATCH(dtype, X, (delta_chunk_prepare_kernel<X><<<dim3(count, H), 256, 0, stream>>>(
      static_cast<const X*>(qkv), ld, static_cast<const X*>(beta), ldb, static_cast<const X*>(decay), lda, a_log, dt_bias, w, v,
      k, pairs, q_factor, totals, table, H, G, D, E, DP, EP, q_scale, unit_eps)));
  if ((status = launch_status()) != 0) return status;
  const dim3 grid(B, H, EP / 16);
#define DISTIE_DELTA_STATES(TILES)                                                                                    \
  delta_chunk_states_kernel<TILES><<<grid, 256, 0, stream>>>(w, v, k, totals, u, states, state, first_chunk, state_slots, H, \
                                                             D, E, EP)
  if (DP == 64) {
    DISTIE_DELTA_STATES(1);
  } else if (DP == 128) {
    DISTIE_DELTA_STATES(2);
  } else {
    DISTIE_DELTA_STATES(4);
  }
#undef DISTIE_DELTA_STATES
  if ((status = launch_status()) != 0) return status;
  DISTIE_DISPATCH(dtype, X, (delta_chunk_outputs_kernel<X><<<dim3(count, H, (E + 63) / 64), 256, 0, stream>>>(
      static_cast<const X*>(qkv), ld, q_factor, pairs, u, states, out, table, H, G, D, E, DP, EP)));
  return launch_status();
}
