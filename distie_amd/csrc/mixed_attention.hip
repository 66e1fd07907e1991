// Attention over the paged cache for layers whose heads see each other's scores: the scores of a query and a key are
// worked out for all heads together, so a workgroup owns every head of a token.
//
//   s_h = cap(q_h . k_(h / (H / G)) * scale) + bias[h][min(i - j, N - 1)]       cap(s) = c tanh(s / c), or s where c is 0
//   s_h <- sum_g mix[h][g] s_g                                                  (no `mix`: s_h)
//   weight_h = exp(s_h) / (exp(sink_h) + sum over the visible keys of exp(s_h)),    out_h = sum of weight_h v
//
// Key j is visible to query i iff j <= i and (i - j < window, or there is no window, or j < keep). Keys and values are
// read through the block table of the token's request; the layouts are those of the other attention kernels (keys
// [pages, kv_heads, P, D], values [pages, kv_heads, D, P]). Scores, mixing, softmax and all sums are float32.
//
// This is the kernel for any types and sizes: one block of four waves a token. A chunk of 64 keys at a time: the waves
// deal the heads among themselves, a lane owns a key; raw scores meet in LDS, are mixed, and the chunk's weights meet in
// LDS again for the sums over the values.
#include "common.h"

namespace {

constexpr int MA_WAVES = 4;
constexpr int MA_LDS_LIMIT = 150 * 1024;

static __host__ __device__ __forceinline__ size_t mixed_lds_floats(int H, int D) {
  return 2 * static_cast<size_t>(H) * D + 2 * static_cast<size_t>(H) * 64 + 3 * static_cast<size_t>(H);
}

template <typename T, typename C>
__global__ void __launch_bounds__(64 * MA_WAVES)
mixed_attention_generic_kernel(const T* __restrict__ q_in, int64_t q_stride, const C* __restrict__ k_cache,
                               const C* __restrict__ v_cache, const int32_t* __restrict__ positions,
                               const int32_t* __restrict__ token_request, const int32_t* __restrict__ block_table,
                               int table_width, const int32_t* __restrict__ table_rows, T* __restrict__ out, int H, int G,
                               int D, int block_size, float scale, int window, int keep, float cap,
                               const float* __restrict__ bias, int bias_len, const float* __restrict__ mix,
                               const float* __restrict__ sinks) {
  extern __shared__ float lds[];
  __shared__ int64_t page_s[64];
  float* q_s = lds;                  // [H][D]
  float* acc = q_s + H * D;          // [H][D]
  float* s_s = acc + H * D;          // [H][64]
  float* p_s = s_s + H * 64;         // [H][64]
  float* m_s = p_s + H * 64;         // [H] running maximum
  float* l_s = m_s + H;              // [H] running sum
  float* a_s = l_s + H;              // [H] what the sums so far are multiplied by
  const int lane = threadIdx.x % 64, wave = threadIdx.x / 64;
  const int64_t t = blockIdx.x;
  const int pos = positions[t];
  const int request = token_request[t];
  const int32_t* table = block_table + static_cast<int64_t>(table_rows != nullptr ? table_rows[request] : request) * table_width;
  for (int i = threadIdx.x; i < H * D; i += blockDim.x) {
    q_s[i] = to_float(q_in[t * q_stride + i]);
    acc[i] = 0.f;
  }
  for (int h = threadIdx.x; h < H; h += blockDim.x) m_s[h] = -INFINITY, l_s[h] = 0.f;
  __syncthreads();
  const int first = window > 0 ? max(0, pos - window + 1) : 0;
  const int group = H / G;
  for (int c = 0; c <= pos; c += 64) {
    if (c >= keep && c + 63 < first) c = first / 64 * 64;         // nothing is visible between the kept keys and the window
    const int key = c + lane;
    const bool seen = key <= pos && (key >= first || key < keep);
    int64_t page = -1;
    if (seen) page = table[key / block_size];
    if (wave == 0) page_s[lane] = page;
    for (int h = wave; h < H; h += MA_WAVES) {
      float s = 0.f;
      if (seen) {
        const C* k = k_cache + ((page * G + h / group) * block_size + key % block_size) * D;
        const float* q = q_s + h * D;
        for (int d = 0; d < D; ++d) s = fmaf(q[d], to_float(k[d]), s);
        s *= scale;
        if (cap > 0.f) s = cap * tanhf(s / cap);
        if (bias != nullptr) s += bias[static_cast<int64_t>(h) * bias_len + min(pos - key, bias_len - 1)];
      }
      s_s[h * 64 + lane] = s;
    }
    __syncthreads();
    for (int h = wave; h < H; h += MA_WAVES) {
      float s = s_s[h * 64 + lane];
      if (mix != nullptr) {
        s = 0.f;
        for (int g = 0; g < H; ++g) s = fmaf(mix[h * H + g], s_s[g * 64 + lane], s);
      }
      const float top = fmaxf(m_s[h], wave_max(seen ? s : -INFINITY));
      const float alpha = top == -INFINITY ? 0.f : expf(m_s[h] - top);
      const float p = seen ? expf(s - top) : 0.f;
      const float sum = wave_sum(p);
      p_s[h * 64 + lane] = p;
      if (lane == 0) {
        l_s[h] = l_s[h] * alpha + sum;
        m_s[h] = top;
        a_s[h] = alpha;
      }
    }
    __syncthreads();
    for (int i = threadIdx.x; i < H * D; i += blockDim.x) {
      const int h = i / D, d = i % D;
      float a = acc[i] * a_s[h];
      for (int j = 0; j < 64; ++j) {
        if (page_s[j] < 0) continue;                              // never a value of a key that is not seen
        a = fmaf(p_s[h * 64 + j], to_float(v_cache[((page_s[j] * G + h / group) * D + d) * block_size + (c + j) % block_size]), a);
      }
      acc[i] = a;
    }
    __syncthreads();
  }
  for (int i = threadIdx.x; i < H * D; i += blockDim.x) {
    const int h = i / D;
    const float sink = sinks != nullptr ? sinks[h] : -INFINITY;
    const float top = fmaxf(m_s[h], sink);
    const float weight = expf(m_s[h] - top);
    out[t * H * D + i] = from_float<T>(acc[i] * (weight / (l_s[h] * weight + (sink == -INFINITY ? 0.f : expf(sink - top)))));
  }
}

}  // namespace

extern "C" int distie_mixed_attention_fits(int H, int D) {
  return H >= 1 && D >= 1 && mixed_lds_floats(H, D) * sizeof(float) <= static_cast<size_t>(MA_LDS_LIMIT) ? 1 : 0;
}

// q: [T, H * D] of `dtype` (rows q_stride apart); out: [T, H * D] of the same; bias: [H, bias_len]; mix: [H, H]; sinks: [H]
extern "C" int distie_mixed_attention_generic(const void* q, int dtype, int64_t q_stride, const void* k_cache,
                                              const void* v_cache, int cache_dtype, const int32_t* positions,
                                              const int32_t* token_request, const int32_t* block_table, int table_width,
                                              const int32_t* table_rows, void* out, int T, int H, int G, int D,
                                              int block_size, float scale, int window, int keep, float cap,
                                              const float* bias, int bias_len, const float* mix, const float* sinks,
                                              hipStream_t stream) {
  if (T <= 0) return 0;
  if (H < 1 || G < 1 || H % G || D < 1 || block_size < 1 || table_width < 1 || window < 0 || keep < 0 ||
      (bias != nullptr && bias_len < 1) || !distie_mixed_attention_fits(H, D) || q_stride < static_cast<int64_t>(H) * D)
    return DISTIE_BAD_ARGUMENT;
  const size_t lds = mixed_lds_floats(H, D) * sizeof(float);
  DISTIE_DISPATCH(dtype, X, DISTIE_DISPATCH(cache_dtype, C, {
    if (lds > 48 * 1024 &&
        hipFuncSetAttribute(reinterpret_cast<const void*>(mixed_attention_generic_kernel<X, C>),
                            hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(lds)) != hipSuccess)
      return DISTIE_BAD_ARGUMENT;
    mixed_attention_generic_kernel<X, C><<<T, 64 * MA_WAVES, lds, stream>>>(
        static_cast<const X*>(q), q_stride, static_cast<const C*>(k_cache), static_cast<const C*>(v_cache), positions,
        token_request, block_table, table_width, table_rows, static_cast<X*>(out), H, G, D, block_size, scale, window, keep,
        cap, bias, bias_len, mix, sinks);
  }));
  return launch_status();
}
