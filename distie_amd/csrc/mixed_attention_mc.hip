// Attention whose heads see each other's scores, bfloat16 on the matrix cores, for one head size (compile with
// -DDISTIE_HEAD_DIM=<a multiple of 32>). What is computed and how keys are read is what mixed_attention.hip says; pages hold
// a multiple of 16 tokens here, so 16 keys that begin at a multiple of 16 lie in one page.
//
//  * mixed_prefill: a workgroup of eight waves owns QT queries of a request and all heads, and walks the visible keys 32 at a
//    time. (1) Raw scores: the columns of a product are 16 (query, head) pairs on one key/value head; column tiles are dealt
//    to the waves. Scale, cap and bias, then into LDS, float32. (2) A wave owns queries: for each, the heads' scores of 16 keys
//    are mixed as a float32 matrix product (heads x heads times heads x keys), masked, and their softmax is carried on; the
//    weights go to LDS in bfloat16. (3) The waves add weights times values to the columns of (1), which they keep.
//  * mixed_decode: one token a request; a workgroup of sixteen waves owns 64 keys of it. Four waves share 16 keys: they score
//    and mix them for all heads, all agree on the maxima, and the sums over the 64 keys go to memory as a partial result.
//  * mixed_reduce: puts a token's partial results together.
#include "common.h"

#ifndef DISTIE_HEAD_DIM
#error "compile with -DDISTIE_HEAD_DIM=<head size>"
#endif
#if DISTIE_HEAD_DIM % 32 != 0 || DISTIE_HEAD_DIM < 32 || DISTIE_HEAD_DIM > 256
#error "head size must be a multiple of 32 up to 256"
#endif

namespace {

constexpr int D = DISTIE_HEAD_DIM;
constexpr float LOG2E = 1.4426950408889634f;
constexpr int LDS_LIMIT = 160 * 1024;

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float floatx4;

struct MixedArgs {
  const bf16_t* q;               // [T, H * D], rows q_stride apart
  int64_t q_stride;
  const bf16_t* k_cache;         // [pages, G, block_size, D]
  const bf16_t* v_cache;         // [pages, G, D, block_size]
  const int32_t* positions;
  const int32_t* cu_q;
  const int32_t* block_table;
  const int32_t* table_rows;     // a request's row of the table (null: its index)
  bf16_t* out;                   // [T, H * D]
  const float* bias;             // [H, bias_len] or null
  const float* mix;              // [H, H] or null
  const float* sinks;            // [H] or null
  float* partial_o;              // decode: [B, splits, H, D]
  float* partial_ml;             // decode: [B, splits, H, 2]
  int table_width, bias_len, requests, H, G, block_size, window, keep, splits, skip_singles, all_single;
  float scale, cap;
};

template <int CTRL>
__device__ __forceinline__ float row_move(float x) {
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, x), CTRL, 0xf, 0xf, true));
}
// over the 16 lanes of a row, the result in all of them (rotations within the row)
__device__ __forceinline__ float row_max(float v) {
  v = fmaxf(v, row_move<0x128>(v));
  v = fmaxf(v, row_move<0x124>(v));
  v = fmaxf(v, row_move<0x122>(v));
  return fmaxf(v, row_move<0x121>(v));
}
__device__ __forceinline__ float row_sum(float v) {
  v += row_move<0x128>(v);
  v += row_move<0x124>(v);
  v += row_move<0x122>(v);
  return v + row_move<0x121>(v);
}

__device__ __forceinline__ float exponential(float x) { return __builtin_amdgcn_exp2f(x * LOG2E); }

// scale, then cap * tanh(s / cap) as cap * (1 - 2 / (e^(2 s / cap) + 1)); `bend` is 2 log2(e) / cap, or 0 without a cap
__device__ __forceinline__ float capped(float s, float scale, float cap, float bend) {
  s *= scale;
  return bend == 0.f ? s : cap - 2.f * cap * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(s * bend) + 1.f);
}

__device__ __forceinline__ int heads_padded(int H) { return (H + 15) / 16 * 16; }

// the mixing matrix into LDS, rows HP + 4 apart, zeros for heads that are not there; no matrix: the heads' own scores
__device__ __forceinline__ void stage_mix(const MixedArgs& p, int HP, float* __restrict__ to) {
  for (int i = threadIdx.x; i < HP * HP; i += blockDim.x) {
    const int h = i / HP, g = i % HP;
    float v = 0.f;
    if (h < p.H && g < p.H) v = p.mix != nullptr ? p.mix[h * p.H + g] : (h == g ? 1.f : 0.f);
    to[h * (HP + 4) + g] = v;
  }
}

// ------------------------------------------------------------------------------------------------ portions of prompts
constexpr int PF_WAVES = 8;
constexpr int KT = 32;           // keys of a step
constexpr int KP = KT + 4;       // floats between the queries of a head's scores
constexpr int PP = KT + 8;       // bfloat16 values between the rows of weights

template <int QT> constexpr int scores_stride() { return QT * KP + 16; }     // between heads: 16 or 48 banks apart

template <int QT>
size_t prefill_lds(int H) {
  const int HP = (H + 15) / 16 * 16;
  return sizeof(float) * (static_cast<size_t>(HP) * scores_stride<QT>() + static_cast<size_t>(HP) * (HP + 4) +
                          2 * static_cast<size_t>(H) * (QT + KT) + 3 * static_cast<size_t>(HP) * QT) +
         sizeof(bf16_t) * static_cast<size_t>(HP) * QT * PP;
}

template <int QT, int NT, bool ONE>                         // ONE: up to 16 heads, one tile of the mixing product
__global__ void __launch_bounds__(64 * PF_WAVES)
mixed_prefill_kernel(MixedArgs p) {
  constexpr int HS = scores_stride<QT>(), BW = QT + KT;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int H = p.H, G = p.G, group = H / G, HP = heads_padded(H), bs = p.block_size;
  bf16_t* P = reinterpret_cast<bf16_t*>(lds);              // [HP * QT][PP]
  float* S = lds + HP * QT * PP / 2;                       // [HP][HS]: head, query, key
  float* M = S + HP * HS;                                  // [HP][HP + 4]
  float* bias_s = M + HP * (HP + 4);                       // [2][H][BW]: bias of distance (pos0 - c) + x - (KT - 1)
  float* m_s = bias_s + 2 * H * BW;                        // [HP][QT]
  float* l_s = m_s + HP * QT;
  float* a_s = l_s + HP * QT;
  const int lane = threadIdx.x % 64, wave = __builtin_amdgcn_readfirstlane(threadIdx.x / 64), i = lane % 16, g = lane / 16;

  // which request's which tile: request b's tiles begin at place cu_q[b] / QT + b
  int count = 0;
  for (int b0 = 0; b0 < p.requests; b0 += 64) {
    const int b = b0 + lane;
    count += __popcll(__ballot(b < p.requests && p.cu_q[min(b, p.requests)] / QT + b <= static_cast<int>(blockIdx.x)));
  }
  const int request = count - 1;
  const int row0 = p.cu_q[request], rows = p.cu_q[request + 1] - row0;
  const int q0 = (static_cast<int>(blockIdx.x) - (row0 / QT + request)) * QT;
  if (q0 >= rows || (p.skip_singles && rows == 1)) return;
  const int nq = min(QT, rows - q0);
  const int64_t t0 = row0 + q0;
  const int pos0 = p.positions[t0];
  const int last = pos0 + nq - 1;
  const int first = p.window > 0 ? max(0, pos0 - p.window + 1) : 0;
  const int keep = p.window > 0 ? p.keep : 0;
  const int32_t* table = p.block_table + static_cast<int64_t>(p.table_rows != nullptr ? p.table_rows[request] : request) * p.table_width;
  const float bend = p.cap > 0.f ? 2.f * LOG2E / p.cap : 0.f;

  stage_mix(p, HP, M);
  for (int x = threadIdx.x; x < (HP - H) * HS; x += blockDim.x) S[H * HS + x] = 0.f;
  for (int x = threadIdx.x; x < HP * QT; x += blockDim.x) m_s[x] = -INFINITY, l_s[x] = 0.f;
  for (int x = threadIdx.x; x < HP * QT * PP / 2; x += blockDim.x) reinterpret_cast<uint32_t*>(P)[x] = 0u;
  // the biases of a step's distances: asked for by `load_bias` (the first two of a thread), in LDS after `stage_bias`
  float bias_held[2] = {0.f, 0.f};
  const auto bias_at = [&](int c, int x) {
    return p.bias[static_cast<int64_t>(x / BW) * p.bias_len + min(max(pos0 - c + x % BW - (KT - 1), 0), p.bias_len - 1)];
  };
  const auto load_bias = [&](int c) {
    if (p.bias == nullptr) return;
#pragma unroll
    for (int k = 0; k < 2; ++k) bias_held[k] = bias_at(c, min(static_cast<int>(threadIdx.x) + k * 64 * PF_WAVES, H * BW - 1));
  };
  const auto stage_bias = [&](int c, int buffer) {
    if (p.bias == nullptr) return;
    float* to = bias_s + buffer * H * BW;
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      const int x = threadIdx.x + k * 64 * PF_WAVES;
      if (x < H * BW) to[x] = bias_held[k];
    }
    for (int x = threadIdx.x + 2 * 64 * PF_WAVES; x < H * BW; x += 64 * PF_WAVES) to[x] = bias_at(c, x);
  };

  // this wave's columns: tile n holds 16 pairs of a query and a head of key/value head kh[n]
  const int tiles = (QT * group + 15) / 16;
  bool have[NT], column[NT];
  int kh[NT], head[NT], query[NT];
  bf16x8 q[NT][D / 32];
  floatx4 o[NT][D / 16];
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    const int tile = wave + PF_WAVES * n;
    have[n] = tile < G * tiles;
    kh[n] = min(tile / tiles, G - 1);
    const int c = tile % tiles * 16 + i;
    query[n] = c % QT;
    column[n] = have[n] && c / QT < group;
    head[n] = kh[n] * group + min(c / QT, group - 1);
    const bf16_t* src = p.q + (t0 + min(query[n], nq - 1)) * p.q_stride + static_cast<int64_t>(head[n]) * D + 8 * g;
#pragma unroll
    for (int s = 0; s < D / 32; ++s) q[n][s] = *reinterpret_cast<const bf16x8*>(src + 32 * s);
#pragma unroll
    for (int d = 0; d < D / 16; ++d) o[n][d] = floatx4{0.f, 0.f, 0.f, 0.f};
  }

  // Where the registers allow it, a step's keys are asked for while the step before is mixed, and its values before its own
  // scores are made: what is left of a trip to memory then hides behind the other phases.
  constexpr bool AHEAD = NT * D <= 128;
  bf16x8 keys[AHEAD ? NT : 1][2][D / 32];
  // the pages of a step's two runs of 16 keys; a run that nobody sees takes the other's (its weights are zero)
  const auto pages_of = [&](int at, int page[2]) {
    bool seen[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int k0 = at + 16 * u;
      seen[u] = k0 <= last && (k0 + 15 >= first || k0 < keep);
      page[u] = seen[u] ? table[k0 / bs] : -1;
    }
    if (!seen[0]) page[0] = page[1];
    if (!seen[1]) page[1] = page[0];
  };
  const auto keys_at = [&](int at, int page, int u, int n) {
    const int k0 = at + 16 * u;
    return p.k_cache + ((static_cast<int64_t>(page) * G + kh[n]) * bs + k0 % bs + i) * D + 8 * g;
  };
  const auto load_keys = [&](int at, const int page[2]) {
    if constexpr (AHEAD) {
#pragma unroll
      for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int u = 0; u < 2; ++u) {
          const bf16_t* src = keys_at(at, page[u], u, n);
#pragma unroll
          for (int s = 0; s < D / 32; ++s) keys[n][u][s] = *reinterpret_cast<const bf16x8*>(src + 32 * s);
        }
    }
  };
  const auto next_step = [&](int c) { return c >= keep && c + KT - 1 < first ? first / KT * KT : c; };
  int c = next_step(0), buffer = 0;
  load_bias(c);
  int page[2], page_next[2];
  pages_of(c, page);                           // (the first step holds key 0 or the window's first: somebody sees it)
  load_keys(c, page);
  int following = next_step(c + KT);
  page_next[0] = page[0], page_next[1] = page[1];
  if (following <= last) pages_of(following, page_next);
  stage_bias(c, buffer);
  __syncthreads();
  // running maxima and sums of this wave's queries, lane (i, g) with heads 4 g .. 4 g + 3 of a tile, for all i alike: in
  // registers where there is one tile, else in m_s and l_s
  constexpr int QW = QT / PF_WAVES;
  float top_of[QW][4], total_of[QW][4];
#pragma unroll
  for (int w = 0; w < QW; ++w)
#pragma unroll
    for (int r = 0; r < 4; ++r) top_of[w][r] = -INFINITY, total_of[w][r] = 0.f;
  float mix_rows[4];                           // ONE: this lane's part of the mixing matrix
#pragma unroll
  for (int s = 0; s < 4; ++s) mix_rows[s] = ONE ? M[i * (HP + 4) + g + 4 * s] : 0.f;
  while (c <= last) {
    bf16x8 values[AHEAD ? NT : 1][D / 16];
    const auto values_at = [&](int n) {
      return p.v_cache + ((static_cast<int64_t>(g < 2 ? page[0] : page[1]) * G + kh[n]) * D + i) * bs + (c + 8 * g) % bs;
    };
    if constexpr (AHEAD) {
#pragma unroll
      for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int d = 0; d < D / 16; ++d)
          values[n][d] = *reinterpret_cast<const bf16x8*>(values_at(n) + static_cast<int64_t>(16 * d) * bs);
    }
    // what the step after the next and the next one will need: pages and biases
    const int later = next_step(following + KT);
    int page_later[2] = {page_next[0], page_next[1]};
    if (later <= last) pages_of(later, page_later);
    if (following <= last) load_bias(following);
    // (1) raw scores of this wave's columns
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      if (!have[n]) continue;
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        const bf16_t* src = keys_at(c, page[u], u, n);
        floatx4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < D / 32; ++s) {
          if constexpr (AHEAD) {
            acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(keys[n][u][s], q[n][s], acc, 0, 0, 0);
          } else {
            acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(src + 32 * s), q[n][s], acc, 0, 0, 0);
          }
        }
        float v[4];
        const float* by_distance = bias_s + (buffer * H + head[n]) * BW + query[n] - (16 * u + 4 * g) + KT - 1;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          v[r] = capped(acc[r], p.scale, p.cap, bend);
          if (p.bias != nullptr) v[r] += by_distance[-r];
        }
        if (column[n]) *reinterpret_cast<float4*>(S + head[n] * HS + query[n] * KP + 16 * u + 4 * g) = float4{v[0], v[1], v[2], v[3]};
      }
    }
    __syncthreads();
    // (2) this wave's queries: mix the heads, mask, carry the softmax on
    if (following <= last) {
      load_keys(following, page_next);
      stage_bias(following, 1 - buffer);
    }
#pragma unroll
    for (int w = 0; w < QW; ++w) {
      const int y = wave + w * PF_WAVES;
      if (y >= nq) break;
      const int pos = pos0 + y;
      const int from = p.window > 0 ? max(0, pos - p.window + 1) : 0;
      const int key_a = c + i, key_b = key_a + 16;
      const bool see_a = key_a <= pos && (key_a >= from || key_a < keep);
      const bool see_b = key_b <= pos && (key_b >= from || key_b < keep);
      const float* scores = S + g * HS + y * KP + i;
      for (int h0 = 0; h0 < (ONE ? 16 : HP); h0 += 16) {
        floatx4 a = {0.f, 0.f, 0.f, 0.f}, b = {0.f, 0.f, 0.f, 0.f};
        if constexpr (ONE) {
#pragma unroll
          for (int s = 0; s < 4; ++s) {
            a = __builtin_amdgcn_mfma_f32_16x16x4f32(mix_rows[s], scores[4 * s * HS], a, 0, 0, 0);
            b = __builtin_amdgcn_mfma_f32_16x16x4f32(mix_rows[s], scores[4 * s * HS + 16], b, 0, 0, 0);
          }
        } else {
          const float* rows_of_m = M + (h0 + i) * (HP + 4) + g;
          for (int s = 0; s < HP; s += 4) {
            const float weight = rows_of_m[s];
            a = __builtin_amdgcn_mfma_f32_16x16x4f32(weight, scores[s * HS], a, 0, 0, 0);
            b = __builtin_amdgcn_mfma_f32_16x16x4f32(weight, scores[s * HS + 16], b, 0, 0, 0);
          }
        }
        float alpha[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float va = see_a ? a[r] : -INFINITY, vb = see_b ? b[r] : -INFINITY;
          const int at = (h0 + 4 * g + r) * QT + y;
          const float old = ONE ? top_of[w][r] : m_s[at];
          const float top = fmaxf(old, row_max(fmaxf(va, vb)));
          const float pa = see_a ? exponential(va - top) : 0.f, pb = see_b ? exponential(vb - top) : 0.f;
          alpha[r] = old == top ? 1.f : exponential(old - top);
          const float total = (ONE ? total_of[w][r] : l_s[at]) * alpha[r] + row_sum(pa + pb);
          if constexpr (ONE) {
            total_of[w][r] = total;
            top_of[w][r] = top;
          } else if (i == 0) {
            m_s[at] = top;
            l_s[at] = total;
          }
          bf16_t* to = P + at * PP + i;
          to[0] = static_cast<bf16_t>(pa);
          to[16] = static_cast<bf16_t>(pb);
        }
        if (i == 0) {
#pragma unroll
          for (int r = 0; r < 4; ++r) a_s[(h0 + 4 * g + r) * QT + y] = alpha[r];
        }
      }
    }
    __syncthreads();
    // (3) weights times values
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      if (!have[n]) continue;
      const int at = head[n] * QT + query[n];
      const float alpha = query[n] < nq ? a_s[at] : 1.f;
      if (__ballot(alpha != 1.f)) {
#pragma unroll
        for (int d = 0; d < D / 16; ++d) o[n][d] *= alpha;
      }
      const bf16x8 weights = *reinterpret_cast<const bf16x8*>(P + at * PP + 8 * g);
#pragma unroll
      for (int d = 0; d < D / 16; ++d) {
        if constexpr (AHEAD) {
          o[n][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(values[n][d], weights, o[n][d], 0, 0, 0);
        } else {
          o[n][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              *reinterpret_cast<const bf16x8*>(values_at(n) + static_cast<int64_t>(16 * d) * bs), weights, o[n][d], 0, 0, 0);
        }
      }
    }
    c = following, following = later;
    page[0] = page_next[0], page[1] = page_next[1];
    page_next[0] = page_later[0], page_next[1] = page_later[1];
    buffer = 1 - buffer;
  }
  if (ONE && i == 0) {
#pragma unroll
    for (int w = 0; w < QW; ++w)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int at = (4 * g + r) * QT + wave + w * PF_WAVES;
        m_s[at] = top_of[w][r];
        l_s[at] = total_of[w][r];
      }
  }
  __syncthreads();
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    if (!column[n] || query[n] >= nq) continue;
    const int at = head[n] * QT + query[n];
    const float sink = p.sinks != nullptr ? p.sinks[head[n]] : -INFINITY;
    const float top = fmaxf(m_s[at], sink);
    const float weight = expf(m_s[at] - top);
    const float inv = weight / (l_s[at] * weight + (sink == -INFINITY ? 0.f : expf(sink - top)));
    bf16_t* dst = p.out + ((t0 + query[n]) * H + head[n]) * D + 4 * g;
#pragma unroll
    for (int d = 0; d < D / 16; ++d) {
      uint32_t bits[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) bits[r] = __builtin_bit_cast(uint16_t, static_cast<bf16_t>(o[n][d][r] * inv));
      *reinterpret_cast<uint2*>(dst + 16 * d) = uint2{bits[0] | (bits[1] << 16), bits[2] | (bits[3] << 16)};
    }
  }
}

// ------------------------------------------------------------------------------------------------ single tokens
constexpr int DC_WAVES = 16;
constexpr int DC_KEYS = 64;
constexpr int DC_RUNS = DC_KEYS / 16;    // runs of 16 keys; DC_WAVES / DC_RUNS waves share a run's heads
constexpr int RD_WAVES = 4;              // of the kernel that puts partial results together
constexpr int DC_SP = DC_KEYS + 16;      // floats between the heads' scores
constexpr int DC_PP = DC_KEYS + 8;       // bfloat16 values between the heads' weights
constexpr int MAX_HEAD_TILES = DC_WAVES / DC_RUNS;

size_t decode_lds(int H) {
  const int HP = (H + 15) / 16 * 16;
  return sizeof(float) * static_cast<size_t>(HP) * (DC_SP + HP + 4 + 2 * DC_RUNS) + sizeof(bf16_t) * static_cast<size_t>(HP) * DC_PP;
}

// which runs of 64 keys the token at `pos` sees: those with kept first keys ahead of the window's, then the window's
struct VisibleRuns {
  int kept, from, total;
  __device__ __forceinline__ VisibleRuns(int pos, int window, int keep) {
    const int first = window > 0 ? max(0, pos - window + 1) : 0;
    kept = window > 0 ? min((min(keep, first) + DC_KEYS - 1) / DC_KEYS, first / DC_KEYS + 1) : 0;
    from = max(first / DC_KEYS, kept);
    total = kept + max(0, pos / DC_KEYS - from + 1);
  }
  __device__ __forceinline__ int run(int index) const { return index < kept ? index : from + index - kept; }
};

__global__ void __launch_bounds__(64 * DC_WAVES)
mixed_decode_kernel(MixedArgs p) {
  constexpr int PARTS = DC_WAVES / DC_RUNS;
  constexpr int AHEAD = 2;                                 // tiles of values a wave asks for before the scores are made
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int H = p.H, G = p.G, group = H / G, HP = heads_padded(H), bs = p.block_size;
  bf16_t* P = reinterpret_cast<bf16_t*>(lds);              // [HP][DC_PP]
  float* S = lds + HP * DC_PP / 2;                         // [HP][DC_SP]
  float* M = S + HP * DC_SP;                               // [HP][HP + 4]
  float* run_top = M + HP * (HP + 4);                      // [DC_RUNS][HP]
  float* run_total = run_top + DC_RUNS * HP;               // [DC_RUNS][HP]
  const int lane = threadIdx.x % 64, wave = __builtin_amdgcn_readfirstlane(threadIdx.x / 64), i = lane % 16, g = lane / 16;
  const int run = wave % DC_RUNS, part = wave / DC_RUNS;
  const int request = blockIdx.y, split = blockIdx.x;
  const int64_t t = p.all_single ? request : p.cu_q[request];
  if (!p.all_single && p.cu_q[request + 1] - t != 1) return;
  const int pos = p.positions[t];
  const VisibleRuns runs(pos, p.window, p.keep);
  if (split >= runs.total) return;
  const int c = runs.run(split) * DC_KEYS;
  const int first = p.window > 0 ? max(0, pos - p.window + 1) : 0;
  const int keep = p.window > 0 ? p.keep : 0;
  const int32_t* table = p.block_table + static_cast<int64_t>(p.table_rows != nullptr ? p.table_rows[request] : request) * p.table_width;
  const float bend = p.cap > 0.f ? 2.f * LOG2E / p.cap : 0.f;
  int page[DC_RUNS], some = 0, mine = -1;
#pragma unroll
  for (int u = 0; u < DC_RUNS; ++u) {
    const int k0 = c + 16 * u;
    const bool seen = k0 <= pos && (k0 + 15 >= first || k0 < keep);
    page[u] = seen ? table[k0 / bs] : -1;
    if (seen) some = page[u];
    if (u == run) mine = page[u];
  }
#pragma unroll
  for (int u = 0; u < DC_RUNS; ++u)
    if (page[u] < 0) page[u] = some;                       // keys that are not seen have weight zero: any page will do
  const int tiles = (group + 15) / 16;                     // column tiles of a key/value head's query heads
  const int k0 = c + 16 * run;
  // (a) raw scores of the run's keys, the column tiles dealt to the run's waves; the values of the first tiles of (c)
  const int value_tiles = G * tiles * (D / 16);
  bf16x8 values[AHEAD][DC_KEYS / 32];
  const auto values_at = [&](int tile, int m) {
    const int d = tile % (D / 16), kh = tile / (D / 16) / tiles;
    const int at = g < 2 ? page[2 * m] : page[2 * m + 1];
    return p.v_cache + ((static_cast<int64_t>(at) * G + kh) * D + 16 * d + i) * bs + (c + 32 * m + 8 * g) % bs;
  };
  for (int kc = part; kc < G * tiles; kc += PARTS) {
    const int kh = kc / tiles, hg = kc % tiles * 16 + i;
    const int head = kh * group + min(hg, group - 1);
    const bf16_t* k = p.k_cache + ((static_cast<int64_t>(mine < 0 ? some : mine) * G + kh) * bs + k0 % bs + i) * D + 8 * g;
    const bf16_t* q = p.q + t * p.q_stride + static_cast<int64_t>(head) * D + 8 * g;
    bf16x8 kf[D / 32], qf[D / 32];
#pragma unroll
    for (int s = 0; s < D / 32; ++s) {
      kf[s] = *reinterpret_cast<const bf16x8*>(k + 32 * s);
      qf[s] = *reinterpret_cast<const bf16x8*>(q + 32 * s);
    }
    float by_distance[4] = {};
    if (p.bias != nullptr) {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        by_distance[r] = p.bias[static_cast<int64_t>(head) * p.bias_len + min(max(pos - (k0 + 4 * g + r), 0), p.bias_len - 1)];
    }
    if (kc == part) {
#pragma unroll
      for (int x = 0; x < AHEAD; ++x)
#pragma unroll
        for (int m = 0; m < DC_KEYS / 32; ++m)
          values[x][m] = *reinterpret_cast<const bf16x8*>(values_at(min(wave + x * DC_WAVES, value_tiles - 1), m));
    }
    floatx4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < D / 32; ++s) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[s], qf[s], acc, 0, 0, 0);
    float v[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) v[r] = capped(acc[r], p.scale, p.cap, bend) + by_distance[r];
    if (hg < group) *reinterpret_cast<float4*>(S + head * DC_SP + 16 * run + 4 * g) = float4{v[0], v[1], v[2], v[3]};
  }
  if (part >= G * tiles) {
#pragma unroll
    for (int x = 0; x < AHEAD; ++x)
#pragma unroll
      for (int m = 0; m < DC_KEYS / 32; ++m)
        values[x][m] = *reinterpret_cast<const bf16x8*>(values_at(min(wave + x * DC_WAVES, value_tiles - 1), m));
  }
  stage_mix(p, HP, M);
  for (int x = threadIdx.x; x < (HP - H) * DC_SP; x += blockDim.x) S[H * DC_SP + x] = 0.f;
  __syncthreads();
  // (b) mixed and masked scores of 16 heads and the run's keys a wave, the maxima of all runs, weights and their sums
  const int key = k0 + i;
  const bool see = mine >= 0 && key <= pos && (key >= first || key < keep);
  const bool mixes = 16 * part < HP;                       // (a wave has one tile of heads at most: PARTS >= MAX_HEAD_TILES)
  floatx4 mixed = {0.f, 0.f, 0.f, 0.f};
  if (mixes) {
    const float* rows_of_m = M + (16 * part + i) * (HP + 4) + g;
    const float* scores = S + g * DC_SP + 16 * run + i;
    for (int s = 0; s < HP; s += 4)
      mixed = __builtin_amdgcn_mfma_f32_16x16x4f32(rows_of_m[s], scores[s * DC_SP], mixed, 0, 0, 0);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      if (!see) mixed[r] = -INFINITY;
      const float top = row_max(mixed[r]);
      if (i == 0) run_top[run * HP + 16 * part + 4 * g + r] = top;
    }
  }
  __syncthreads();
  if (mixes) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int head = 16 * part + 4 * g + r;
      float top = run_top[head];
#pragma unroll
      for (int u = 1; u < DC_RUNS; ++u) top = fmaxf(top, run_top[u * HP + head]);
      const float weight = see ? exponential(mixed[r] - top) : 0.f;
      const float total = row_sum(weight);
      P[head * DC_PP + 16 * run + i] = static_cast<bf16_t>(weight);
      if (i == 0) run_total[run * HP + head] = total;
    }
  }
  __syncthreads();
  // (c) the partial result
  const int64_t place = (static_cast<int64_t>(request) * p.splits + split) * H;
  for (int h = threadIdx.x; h < H; h += blockDim.x) {
    float top = run_top[h], total = run_total[h];
#pragma unroll
    for (int u = 1; u < DC_RUNS; ++u) top = fmaxf(top, run_top[u * HP + h]), total += run_total[u * HP + h];
    p.partial_ml[(place + h) * 2] = top;
    p.partial_ml[(place + h) * 2 + 1] = total;
  }
  const auto finish = [&](int tile, const bf16x8 v[DC_KEYS / 32]) {
    const int d = tile % (D / 16), kc = tile / (D / 16), kh = kc / tiles, hg = kc % tiles * 16 + i;
    const int head = kh * group + min(hg, group - 1);
    floatx4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int m = 0; m < DC_KEYS / 32; ++m)
      acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v[m], *reinterpret_cast<const bf16x8*>(P + head * DC_PP + 32 * m + 8 * g), acc, 0, 0, 0);
    if (hg < group)
      *reinterpret_cast<float4*>(p.partial_o + (place + head) * D + 16 * d + 4 * g) = float4{acc[0], acc[1], acc[2], acc[3]};
  };
#pragma unroll
  for (int x = 0; x < AHEAD; ++x)
    if (wave + x * DC_WAVES < value_tiles) finish(wave + x * DC_WAVES, values[x]);
  for (int tile = wave + AHEAD * DC_WAVES; tile < value_tiles; tile += DC_WAVES) {
    bf16x8 v[DC_KEYS / 32];
#pragma unroll
    for (int m = 0; m < DC_KEYS / 32; ++m) v[m] = *reinterpret_cast<const bf16x8*>(values_at(tile, m));
    finish(tile, v);
  }
}

// one block a (request, head): the waves deal the partial results, a lane owns dimensions lane, lane + 64, ...
__global__ void __launch_bounds__(64 * RD_WAVES)
mixed_reduce_kernel(MixedArgs p) {
  __shared__ float sums[RD_WAVES][D], tops[RD_WAVES], totals[RD_WAVES];
  const int lane = threadIdx.x % 64, wave = threadIdx.x / 64;
  const int request = blockIdx.x, head = blockIdx.y;
  const int64_t t = p.all_single ? request : p.cu_q[request];
  if (!p.all_single && p.cu_q[request + 1] - t != 1) return;
  const VisibleRuns runs(p.positions[t], p.window, p.keep);
  const int64_t place = static_cast<int64_t>(request) * p.splits * p.H + head;
  float top = -INFINITY, total = 0.f, acc[(D + 63) / 64];
#pragma unroll
  for (int x = 0; x < (D + 63) / 64; ++x) acc[x] = 0.f;
  for (int s = wave; s < runs.total; s += RD_WAVES) top = fmaxf(top, p.partial_ml[(place + static_cast<int64_t>(s) * p.H) * 2]);
  if (lane == 0) tops[wave] = top;
  __syncthreads();
  const float sink = p.sinks != nullptr ? p.sinks[head] : -INFINITY;
  top = sink;
#pragma unroll
  for (int w = 0; w < RD_WAVES; ++w) top = fmaxf(top, tops[w]);
  for (int s = wave; s < runs.total; s += RD_WAVES) {
    const int64_t at = place + static_cast<int64_t>(s) * p.H;
    const float weight = expf(p.partial_ml[at * 2] - top);
    total += p.partial_ml[at * 2 + 1] * weight;
#pragma unroll
    for (int x = 0; x < (D + 63) / 64; ++x)
      if (lane + 64 * x < D) acc[x] += p.partial_o[at * D + lane + 64 * x] * weight;
  }
  if (lane == 0) totals[wave] = total;
#pragma unroll
  for (int x = 0; x < (D + 63) / 64; ++x)
    if (lane + 64 * x < D) sums[wave][lane + 64 * x] = acc[x];
  __syncthreads();
  float all = sink == -INFINITY ? 0.f : expf(sink - top);
#pragma unroll
  for (int w = 0; w < RD_WAVES; ++w) all += totals[w];
  for (int d = threadIdx.x; d < D; d += blockDim.x) {
    float v = 0.f;
#pragma unroll
    for (int w = 0; w < RD_WAVES; ++w) v += sums[w][d];
    p.out[(t * p.H + head) * D + d] = static_cast<bf16_t>(v / all);
  }
}

int column_tiles(int H, int G, int QT) { return G * ((QT * (H / G) + 15) / 16); }

// the most column tiles a wave of the prefill kernel may own: their sums stay in its registers
constexpr int MAX_TILES = 512 / D < 1 ? 1 : (512 / D > 8 ? 8 : 512 / D);

bool prefill_fits(int H, int G, int QT) {
  return (column_tiles(H, G, QT) + PF_WAVES - 1) / PF_WAVES <= MAX_TILES &&
         (QT == 16 ? prefill_lds<16>(H) : prefill_lds<8>(H)) <= static_cast<size_t>(LDS_LIMIT);
}

template <int QT, int NT, bool ONE>
int launch_prefill(const MixedArgs& p, int blocks, hipStream_t stream) {
  const size_t lds = prefill_lds<QT>(p.H);
  if (lds > 48 * 1024 && hipFuncSetAttribute(reinterpret_cast<const void*>(mixed_prefill_kernel<QT, NT, ONE>),
                                             hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(lds)) != hipSuccess)
    return DISTIE_BAD_ARGUMENT;
  mixed_prefill_kernel<QT, NT, ONE><<<blocks, 64 * PF_WAVES, lds, stream>>>(p);
  return launch_status();
}

template <int QT, bool ONE>
int launch_prefill_tiles(const MixedArgs& p, int blocks, hipStream_t stream) {
  const int each = (column_tiles(p.H, p.G, QT) + PF_WAVES - 1) / PF_WAVES;
  if (each == 1) return launch_prefill<QT, 1, ONE>(p, blocks, stream);
  if constexpr (MAX_TILES >= 2)
    if (each == 2) return launch_prefill<QT, 2, ONE>(p, blocks, stream);
  if constexpr (MAX_TILES >= 4)
    if (each <= 4) return launch_prefill<QT, 4, ONE>(p, blocks, stream);
  if constexpr (MAX_TILES >= 8)
    if (each <= 8) return launch_prefill<QT, 8, ONE>(p, blocks, stream);
  return DISTIE_BAD_ARGUMENT;
}

}  // namespace

extern "C" int distie_mixed_head_dim() { return D; }

// whether the kernels here take H query heads on G key/value heads: 16 or 8 (queries of a prefill workgroup), or 0
extern "C" int distie_mixed_fits(int H, int G) {
  if (H < 1 || G < 1 || H % G || H > 16 * MAX_HEAD_TILES || decode_lds(H) > static_cast<size_t>(LDS_LIMIT)) return 0;
  return prefill_fits(H, G, 16) ? 16 : (prefill_fits(H, G, 8) ? 8 : 0);
}

extern "C" int distie_mixed_decode_keys() { return DC_KEYS; }

// prefill: T rows of B requests in workgroups of `queries` (8 or 16); `decode`: the requests that bring one token (2: all do,
// row b is request b's), `splits` partial results each (at least as many as runs of 64 keys any of them sees)
extern "C" int distie_mixed_attention_bf16(const void* q, int64_t q_stride, const void* k_cache, const void* v_cache,
                                           const int32_t* positions, const int32_t* cu_q, const int32_t* block_table,
                                           int table_width, const int32_t* table_rows, void* out, int T, int B, int H, int G,
                                           int block_size, float scale, int window, int keep, float cap, const float* bias,
                                           int bias_len, const float* mix, const float* sinks, int prefill, int queries,
                                           int decode, int splits, float* partial_o, float* partial_ml, hipStream_t stream) {
  if (T <= 0 || B <= 0) return 0;
  if (!distie_mixed_fits(H, G) || block_size < 16 || block_size % 16 || table_width < 1 || window < 0 || keep < 0 ||
      q_stride % 8 || (bias != nullptr && bias_len < 1) || reinterpret_cast<uintptr_t>(q) % 16 ||
      reinterpret_cast<uintptr_t>(k_cache) % 16 || reinterpret_cast<uintptr_t>(v_cache) % 16 ||
      reinterpret_cast<uintptr_t>(out) % 16 || !(scale > 0.f))
    return DISTIE_BAD_ARGUMENT;
  MixedArgs p;
  p.q = static_cast<const bf16_t*>(q), p.q_stride = q_stride;
  p.k_cache = static_cast<const bf16_t*>(k_cache), p.v_cache = static_cast<const bf16_t*>(v_cache);
  p.positions = positions, p.cu_q = cu_q, p.block_table = block_table, p.table_rows = table_rows;
  p.out = static_cast<bf16_t*>(out), p.bias = bias, p.mix = mix, p.sinks = sinks;
  p.partial_o = partial_o, p.partial_ml = partial_ml;
  p.table_width = table_width, p.bias_len = bias_len, p.requests = B, p.H = H, p.G = G, p.block_size = block_size;
  p.window = window, p.keep = keep, p.splits = splits, p.skip_singles = decode ? 1 : 0;
  p.all_single = decode == 2 ? 1 : 0;
  p.scale = scale, p.cap = cap;
  if (decode) {
    if (splits < 1 || splits > 65535 || B > 65535 || H > 65535 || partial_o == nullptr || partial_ml == nullptr ||
        reinterpret_cast<uintptr_t>(partial_o) % 16)
      return DISTIE_BAD_ARGUMENT;
    const size_t lds = decode_lds(H);
    if (lds > 48 * 1024 && hipFuncSetAttribute(reinterpret_cast<const void*>(mixed_decode_kernel),
                                               hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(lds)) != hipSuccess)
      return DISTIE_BAD_ARGUMENT;
    mixed_decode_kernel<<<dim3(splits, B), 64 * DC_WAVES, lds, stream>>>(p);
    int status = launch_status();
    if (status != 0) return status;
    mixed_reduce_kernel<<<dim3(B, H), 64 * RD_WAVES, 0, stream>>>(p);
    if ((status = launch_status()) != 0) return status;
  }
  if (prefill) {
    if ((queries != 8 && queries != 16) || !prefill_fits(H, G, queries)) return DISTIE_BAD_ARGUMENT;
    const int blocks = T / queries + B + 1;
    if (H <= 16)
      return queries == 16 ? launch_prefill_tiles<16, true>(p, blocks, stream) : launch_prefill_tiles<8, true>(p, blocks, stream);
    return queries == 16 ? launch_prefill_tiles<16, false>(p, blocks, stream)
                         : launch_prefill_tiles<8, false>(p, blocks, stream);
  }
  return 0;
}
