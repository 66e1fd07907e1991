// What the kernels on packed weight copies share: vector types of the matrix cores' operands, the tile of
// a packed copy, and the description of the q/k/v epilogue.
#pragma once

#include "common.h"

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float floatx4;

#define PK_TILE 512         // elements of a tile: 16 rows x 32 k, in lane order
#define PK_PLAIN 0
#define PK_GATED 1
#define PK_ROTARY 2

struct RotaryOut {
  const float2* table;        // [M, D / 2] cosine and sine of each token's angles
  const int32_t* slots;       // [M] place of each token in the cache
  bf16_t* k_cache;            // [pages, kv_heads, block_size, D]
  bf16_t* v_cache;            // [pages, kv_heads, D, block_size]
  int heads, kv_heads, dim, block_size, write;
  int act;                    // gated products only: the activation on the gate (see gate_activation)
  float limit, slope, up_shift;      // of the clamped one (see gated_value)
};

// The activation on the gate of a gated product: 0 silu; else 1 + the kind as `distie_activation` numbers them
// (1: the square of max(z, 0), 3: the tanh form of gelu, 4: max(z, 0)). The C interface takes it in the bits above
// the low eight of its `gated` / `mode` argument.
static __device__ __forceinline__ float gate_activation(float z, int act) {
  if (act == 0 || act == 2) return z / (1.f + expf(-z));
  if (act == 3) return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
  const float p = fmaxf(z, 0.f);
  return act == 1 ? p * p : p;
}

// gate and up of one hidden value put together. act 5: g = min(gate, limit), u = clamp(up, -limit, limit),
// g * sigmoid(slope * g) * (u + up_shift); else the activation of the gate times up.
static __device__ __forceinline__ float gated_value(float gate, float up, int act, float limit, float slope, float up_shift) {
  if (act != 5) return gate_activation(gate, act) * up;
  const float g = fminf(gate, limit), u = fminf(fmaxf(up, -limit), limit);
  return g / (1.f + expf(-slope * g)) * (u + up_shift);
}

static __device__ __forceinline__ uint2 pack_bf16x4(const float v[4]) {
  uint32_t h[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) h[i] = __builtin_bit_cast(uint16_t, static_cast<bf16_t>(v[i]));
  return uint2{h[0] | (h[1] << 16), h[2] | (h[3] << 16)};
}
