// Norms in groups around a residual sum that is averaged over the depth of the model. Everything is float32: the
// statistics, the residual and what is kept of every layer.
#include "common.h"
#include "vector_values.h"

namespace {

// One row a block:
//   y = delta / sqrt(mean over the column's group(delta^2) + eps) * weight        (`groups` equal runs of columns)
//   x = residual_in + y                                                            (null: x = y)
//   with `weights` (float32 [index + 2]): rest[index] = x;  x = sum_j weights[j] X_j,  X_0 = first, X_(j+1) = rest[j]
//   residual_out = x (null: kept nowhere);  out = x in its own precision (null: nobody reads it)
// SHIFT, for steps of one row a request: out is [mixes, T, C] instead, out[m] = h + (before - h) * mu[m] with h = x in out's
// precision and `before` the request's row of `state` (float32 [slots, C], row state_slots[row]), which h replaces.
// delta may be partial sums (slices that lie `stride` elements apart, added in order). A thread keeps Q runs of V columns
// in registers; everything it reads is asked for before the first barrier. The sums of squares of the runs wait in LDS, a
// wave adds up those of a group in an order that only the sizes decide.
constexpr int SHIFT_MIXES = 8;

template <int V, int Q, bool SHIFT, typename A, typename O>
__global__ void __launch_bounds__(1024)
group_chain_kernel(const A* __restrict__ delta, int slices, int64_t stride, const float* __restrict__ weight, float eps,
                   int groups, const float* residual_in, float* residual_out, const float* __restrict__ first, float* rest,
                   int index, const float* __restrict__ weights, O* __restrict__ out, int C, int64_t layer_stride,
                   const float* __restrict__ mu, int mixes, float* __restrict__ state,
                   const int32_t* __restrict__ state_slots) {
  extern __shared__ float lds[];
  const int runs = C / V, per_group = runs / groups;
  float* squares = lds;                       // [runs]
  float* scale = lds + runs;                  // [groups]
  const int64_t base = static_cast<int64_t>(blockIdx.x) * C;
  float y[Q][V], x[Q][V], sum[Q][V];
  float before[SHIFT ? Q : 1][V], own_mu[SHIFT && Q == 1 ? SHIFT_MIXES : 1][V];
  float* own = nullptr;
  if constexpr (SHIFT) {
    own = state + static_cast<int64_t>(state_slots[blockIdx.x]) * C;
#pragma unroll
    for (int q = 0; q < Q; ++q) {
      const int run = threadIdx.x + q * blockDim.x;
      if (run < runs) load_values<V>(own + static_cast<int64_t>(run) * V, before[q]);
    }
    if constexpr (Q == 1) {
      if (static_cast<int>(threadIdx.x) < runs) {
#pragma unroll
        for (int m = 0; m < SHIFT_MIXES; ++m)
          if (m < mixes) load_values<V>(mu + static_cast<int64_t>(m) * C + threadIdx.x * V, own_mu[m]);
      }
    }
  }
#pragma unroll
  for (int q = 0; q < Q; ++q) {
    const int run = threadIdx.x + q * blockDim.x;
#pragma unroll
    for (int k = 0; k < V; ++k) y[q][k] = 0.f, x[q][k] = 0.f, sum[q][k] = 0.f;
    if (run >= runs) continue;
    const int64_t at = base + static_cast<int64_t>(run) * V;
    sum_values<V>(delta + at, slices, stride, y[q]);
    if (residual_in != nullptr) load_values<V>(residual_in + at, x[q]);
  }
  if (weights != nullptr) {
    const float w0 = weights[0];
#pragma unroll
    for (int q = 0; q < Q; ++q) {
      const int run = threadIdx.x + q * blockDim.x;
      if (run >= runs) continue;
      const int64_t at = base + static_cast<int64_t>(run) * V;
      float v[V];
      load_values<V>(first + at, v);
#pragma unroll
      for (int k = 0; k < V; ++k) sum[q][k] = w0 * v[k];
      for (int j = 0; j < index; j += 8) {
        float a[8][V];
#pragma unroll
        for (int u = 0; u < 8; ++u) load_values<V>(rest + min(j + u, index - 1) * layer_stride + at, a[u]);
#pragma unroll
        for (int u = 0; u < 8; ++u)
          if (j + u < index) {
            const float w = weights[j + u + 1];
#pragma unroll
            for (int k = 0; k < V; ++k) sum[q][k] += w * a[u][k];
          }
      }
    }
  }
#pragma unroll
  for (int q = 0; q < Q; ++q) {
    const int run = threadIdx.x + q * blockDim.x;
    if (run >= runs) continue;
    float s = 0.f;
#pragma unroll
    for (int k = 0; k < V; ++k) s += y[q][k] * y[q][k];
    squares[run] = s;
  }
  __syncthreads();
  const int lane = threadIdx.x % 64, waves = blockDim.x / 64;
  for (int g = threadIdx.x / 64; g < groups; g += waves) {
    float s = 0.f;
    for (int r = lane; r < per_group; r += 64) s += squares[g * per_group + r];
    s = wave_sum(s);
    if (lane == 0) scale[g] = 1.f / sqrtf(s / (per_group * V) + eps);
  }
  __syncthreads();
  const float last = weights != nullptr ? weights[index + 1] : 0.f;
#pragma unroll
  for (int q = 0; q < Q; ++q) {
    const int run = threadIdx.x + q * blockDim.x;
    if (run >= runs) continue;
    const int64_t at = base + static_cast<int64_t>(run) * V;
    const float r = scale[run / per_group];
    float w[V];
    load_values<V>(weight + static_cast<int64_t>(run) * V, w);
#pragma unroll
    for (int k = 0; k < V; ++k) x[q][k] += y[q][k] * r * w[k];
    if (weights != nullptr) {
      store_values<V>(rest + index * layer_stride + at, x[q]);
#pragma unroll
      for (int k = 0; k < V; ++k) x[q][k] = sum[q][k] + last * x[q][k];
    }
    if (residual_out != nullptr) store_values<V>(residual_out + at, x[q]);
    if constexpr (SHIFT) {
      float h[V], mixed[V];
#pragma unroll
      for (int k = 0; k < V; ++k) h[k] = to_float(from_float<O>(x[q][k]));
      store_values<V>(own + static_cast<int64_t>(run) * V, h);
#pragma unroll
      for (int m = 0; m < SHIFT_MIXES; ++m) {
        if (m >= mixes) break;
        float w[V];
        if constexpr (Q == 1) {
#pragma unroll
          for (int k = 0; k < V; ++k) w[k] = own_mu[m][k];
        } else {
          load_values<V>(mu + static_cast<int64_t>(m) * C + static_cast<int64_t>(run) * V, w);
        }
#pragma unroll
        for (int k = 0; k < V; ++k) mixed[k] = h[k] + (before[q][k] - h[k]) * w[k];
        store_values<V>(out + m * layer_stride + at, mixed);
      }
    } else {
      if (out != nullptr) store_values<V>(out + at, x[q]);
    }
  }
}

}  // namespace

// delta: [T, C] of `dtype`, or `slices` float32 partial sums [slices, T, C]; rest: [layers, T, C]; mu null: out is [T, C],
// else [mixes, T, C] (see SHIFT above)
extern "C" int distie_group_chain(const void* delta, int dtype, int slices, const float* weight, float eps, int groups,
                                  const float* residual_in, float* residual_out, const float* first, float* rest, int index,
                                  const float* weights, void* out, int out_dtype, int T, int C, const float* mu, int mixes,
                                  float* state, const int32_t* state_slots, hipStream_t stream) {
  if (T <= 0) return 0;
  if (C < 1 || groups < 1 || C % groups || delta == nullptr || weight == nullptr || slices < 1 ||
      (slices > 1 && dtype != DISTIE_F32) || !(eps >= 0.f) || (residual_out == nullptr && out == nullptr) ||
      (mu != nullptr && (mixes < 1 || mixes > SHIFT_MIXES || state == nullptr || state_slots == nullptr || out == nullptr)) ||
      (weights != nullptr && (first == nullptr || rest == nullptr || index < 0 || residual_in == nullptr)))
    return DISTIE_BAD_ARGUMENT;
  const int64_t stride = static_cast<int64_t>(T) * C;
  const auto aligned = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  const bool wide = (C / groups) % 4 == 0 && aligned(delta) && aligned(weight) && aligned(residual_in) &&
                    aligned(residual_out) && aligned(first) && aligned(rest) && aligned(out) && aligned(mu) && aligned(state);
  const int runs = wide ? C / 4 : C;
  const size_t lds = static_cast<size_t>(runs + groups) * sizeof(float);
  if (lds > 48 * 1024) return DISTIE_BAD_ARGUMENT;
  const int threads = runs > 512 ? 1024 : (runs > 256 ? 512 : (runs > 128 ? 256 : (runs > 64 ? 128 : 64)));
  const int each = (runs + threads - 1) / threads;
  if (out == nullptr) out_dtype = DISTIE_F32;
#define DISTIE_GROUP_CHAIN_AS(V, Q, SHIFT)                                                                             \
  DISTIE_DISPATCH(dtype, A, DISTIE_DISPATCH(out_dtype, O, (                                                             \
      group_chain_kernel<V, Q, SHIFT, A, O><<<T, threads, lds, stream>>>(                                               \
          static_cast<const A*>(delta), slices, stride, weight, eps, groups, residual_in, residual_out, first, rest,    \
          index, weights, static_cast<O*>(out), C, stride, mu, mixes, state, state_slots))))
#define DISTIE_GROUP_CHAIN(V, Q)          \
  if (mu != nullptr) {                    \
    DISTIE_GROUP_CHAIN_AS(V, Q, true);    \
  } else {                                \
    DISTIE_GROUP_CHAIN_AS(V, Q, false);   \
  }
  if (wide) {
    if (each == 1) {
      DISTIE_GROUP_CHAIN(4, 1);
    } else if (each == 2) {
      DISTIE_GROUP_CHAIN(4, 2);
    } else if (each <= 4) {
      DISTIE_GROUP_CHAIN(4, 4);
    } else {
      return DISTIE_BAD_ARGUMENT;
    }
  } else {
    if (each <= 2) {
      DISTIE_GROUP_CHAIN(1, 2);
    } else if (each <= 8) {
      DISTIE_GROUP_CHAIN(1, 8);
    } else {
      return DISTIE_BAD_ARGUMENT;
    }
  }
#undef DISTIE_GROUP_CHAIN
#undef DISTIE_GROUP_CHAIN_AS
  return launch_status();
}
