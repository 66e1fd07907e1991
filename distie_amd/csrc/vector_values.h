// Reads and writes of several neighbouring values by one thread, as floats.
#pragma once

#include "common.h"

// V values at p as floats: V = 4 takes one 16-byte (float32) or 8-byte (bfloat16) load, V = 8 two or one of 16 bytes
template <int V, typename T>
__device__ __forceinline__ void load_values(const T* __restrict__ p, float out[V]) {
  if constexpr (V == 8 && sizeof(T) == 4) {
    load_values<4>(p, out);
    load_values<4>(p + 4, out + 4);
  } else if constexpr (V == 8) {
    const uint4 v = *reinterpret_cast<const uint4*>(p);
    const uint32_t w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
    for (int k = 0; k < 4; ++k) out[2 * k] = __uint_as_float(w[k] << 16), out[2 * k + 1] = __uint_as_float(w[k] & 0xffff0000u);
  } else if constexpr (V == 4 && sizeof(T) == 4) {
    const float4 v = *reinterpret_cast<const float4*>(p);
    out[0] = v.x, out[1] = v.y, out[2] = v.z, out[3] = v.w;
  } else if constexpr (V == 4) {
    const uint2 v = *reinterpret_cast<const uint2*>(p);
    out[0] = __uint_as_float(v.x << 16), out[1] = __uint_as_float(v.x & 0xffff0000u);
    out[2] = __uint_as_float(v.y << 16), out[3] = __uint_as_float(v.y & 0xffff0000u);
  } else {
#pragma unroll
    for (int k = 0; k < V; ++k) out[k] = to_float(p[k]);
  }
}

template <int V, typename T>
__device__ __forceinline__ void store_values(T* __restrict__ p, const float v[V]) {
  const auto word = [](float lo, float hi) {
    return static_cast<uint32_t>(__builtin_bit_cast(uint16_t, static_cast<bf16_t>(lo))) |
           (static_cast<uint32_t>(__builtin_bit_cast(uint16_t, static_cast<bf16_t>(hi))) << 16);
  };
  if constexpr (V == 8 && sizeof(T) == 4) {
    store_values<4>(p, v);
    store_values<4>(p + 4, v + 4);
  } else if constexpr (V == 8) {
    *reinterpret_cast<uint4*>(p) = uint4{word(v[0], v[1]), word(v[2], v[3]), word(v[4], v[5]), word(v[6], v[7])};
  } else if constexpr (V == 4 && sizeof(T) == 4) {
    *reinterpret_cast<float4*>(p) = float4{v[0], v[1], v[2], v[3]};
  } else if constexpr (V == 4) {
    *reinterpret_cast<uint2*>(p) = uint2{word(v[0], v[1]), word(v[2], v[3])};
  } else {
#pragma unroll
    for (int k = 0; k < V; ++k) p[k] = from_float<T>(v[k]);
  }
}

// the sum of `slices` vectors that lie `stride` elements apart, added in order; eight slices' loads under way together
template <int V, typename T>
__device__ __forceinline__ void sum_values(const T* __restrict__ p, int slices, int64_t stride, float out[V]) {
  load_values<V>(p, out);
  for (int s = 1; s < slices; s += 8) {
    float a[8][V];
#pragma unroll
    for (int u = 0; u < 8; ++u) load_values<V>(p + min(s + u, slices - 1) * stride, a[u]);
#pragma unroll
    for (int u = 0; u < 8; ++u)
      if (s + u < slices) {
#pragma unroll
        for (int k = 0; k < V; ++k) out[k] += a[u][k];
      }
  }
}
