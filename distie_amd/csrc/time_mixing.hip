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
  const int b = token_request[t];
  const int64_t first = cu_q[b];
  float h[V], before[V];
  load_values<V>(x + t * C + c, h);
  if (t > first) {
    load_values<V>(x + (t - 1) * C + c, before);
  } else {
    float* own = state + static_cast<int64_t>(state_slots[b]) * C + c;
    const int64_t last = cu_q[b + 1] - 1;
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
  const int first = cu_q[b], last = cu_q[b + 1];
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
    for (int i = sub; i < rank; i += SUB) z += up_row[i] * low_s[i];
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

// tanh of a [T, N] float32 view (rows `ld` apart) into a dense tensor
extern "C" int distie_tanh_f32(const float* in, int64_t ld, float* out, int T, int N, hipStream_t stream) {
  if (T <= 0) return 0;
  if (N < 1 || ld < N) return DISTIE_BAD_ARGUMENT;
  const int64_t blocks = (static_cast<int64_t>(T) * N + 255) / 256;
  if (blocks > 0x7fffffff) return DISTIE_BAD_ARGUMENT;
  tanh_f32_kernel<<<static_cast<unsigned>(blocks), 256, 0, stream>>>(in, ld, out, N, T);
  return launch_status();
}
