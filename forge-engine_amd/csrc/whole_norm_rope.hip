// From the projection's output to queries and cached keys and values, for attention that
// normalises q and k over the whole projection: one block per token, or, in a step of few tokens, one
// per token and head.
//   q <- q / sqrt(mean over all heads and dims of q^2 + eps) * w_q      (w_q as long as q; k likewise)
//   the first R dims of every head turn by the token's position: dim i < R/2 pairs with i + R/2,
//   (a, b) -> (a c - b s, b c + a s) with c = magnitude cos(p f_i), s = magnitude sin(p f_i)
//   q into q_out [T, Hq D]; k into pages [page][kv head][slot][D]; v into pages transposed
//   [page][kv head][Dv][slot].
// With write_kv = 0 the row holds q only (a layer that reads another layer's keys and values).
// A bias (float32, over the whole of [q | k | v]) is added to the projection first, if there is one.  Cached rows may
// be wider than a head (key_row, value_row: sizes that the matrix-core attention takes): q and key rows are then
// filled up with zeros, the rest of a value's dims is left alone.
// float32 inside, one rounding at the stores.
#include "common.h"

template <typename T>
__global__ __launch_bounds__(256) void whole_norm_rope_kernel(
    const T* __restrict__ qkv, size_t stride, const float* __restrict__ bias, const float* __restrict__ q_weight,
    const float* __restrict__ k_weight, const float* __restrict__ inv_freq, const int* __restrict__ positions, const int* __restrict__ token_seq,
    const int* __restrict__ block_table, int table_stride, T* __restrict__ key_pages, T* __restrict__ value_pages,
    T* __restrict__ q_out, int q_heads, int kv_heads, int D, int Dv, int R, float eps, float magnitude, int write_kv,
    int block_size, int num_blocks, int key_row, int value_row) {
  __shared__ float cs[128], sn[128];
  __shared__ float scratch[16];
  const int t = blockIdx.x, tid = threadIdx.x;
  const int pos = positions[t];
  const int half = R / 2;
  for (int j = tid; j < half; j += 256) {
    float s, c;
    sincosf((float)pos * inv_freq[j], &s, &c);
    cs[j] = c * magnitude;
    sn[j] = s * magnitude;
  }
  const T* row = qkv + (size_t)t * stride;
  const int q_size = q_heads * D, kv_size = kv_heads * D;
  const float* q_bias = bias;
  const float* k_bias = bias ? bias + q_size : nullptr;
  const float* v_bias = bias ? k_bias + kv_size : nullptr;
  auto biased = [](const T* x, const float* b, int e) { return b ? load_as_float(x + e) + b[e] : load_as_float(x + e); };
  float sq = 0.f, sk = 0.f;
  for (int e = tid; e < q_size; e += 256) {
    const float v = biased(row, q_bias, e);
    sq = fmaf(v, v, sq);
  }
  if (write_kv)
    for (int e = tid; e < kv_size; e += 256) {
      const float v = biased(row + q_size, k_bias, e);
      sk = fmaf(v, v, sk);
    }
  const float inv_q = 1.f / sqrtf(block_sum<true>(sq, scratch) / (float)q_size + eps);
  const float inv_k = write_kv ? 1.f / sqrtf(block_sum(sk, scratch) / (float)kv_size + eps) : 0.f;
  // block_sum's barriers also make cs and sn visible

  auto turned = [&](const T* x, const float* b, const float* w, float inv, int e, int d) {
    float v = biased(x, b, e) * inv * w[e];
    if (d < R) {
      const bool low = d < half;
      const int j = low ? d : d - half;
      const int pe = low ? e + half : e - half;
      const float partner = biased(x, b, pe) * inv * w[pe];
      v = low ? v * cs[j] - partner * sn[j] : v * cs[j] + partner * sn[j];
    }
    return v;
  };

  // Units of work: the q heads, then the k heads, then the v heads.  A launch of many tokens gives a block
  // all units of its token; one of few tokens spreads them over blockIdx.y (every block forms the sums of
  // squares for itself), so that a step of a few single tokens still fills some of the chip.
  const int units = q_heads + (write_kv ? 2 * kv_heads : 0);
  int page = -1, slot = 0;
  if (write_kv) {
    const int seq = token_seq[t];
    page = block_table[(size_t)seq * table_stride + pos / block_size];
    if (page < 0 || page >= num_blocks) page = -1;
    slot = pos % block_size;
  }
  T* qrow = q_out + (size_t)t * q_heads * key_row;
  const T* krow = row + q_size;
  const T* vrow = krow + kv_size;
  // ranges are of heads
  auto q_range = [&](int begin, int end) {
    for (int f = begin * key_row + tid; f < end * key_row; f += 256) {
      const int h = f / key_row, d = f - h * key_row;
      store_from_float(qrow + f, d < D ? turned(row, q_bias, q_weight, inv_q, h * D + d, d) : 0.f);
    }
  };
  auto k_range = [&](int begin, int end) {
    for (int f = begin * key_row + tid; f < end * key_row; f += 256) {
      const int h = f / key_row, d = f - h * key_row;
      store_from_float(key_pages + (((size_t)page * kv_heads + h) * block_size + slot) * key_row + d,
                       d < D ? turned(krow, k_bias, k_weight, inv_k, h * D + d, d) : 0.f);
    }
  };
  auto v_range = [&](int begin, int end) {
    for (int e = begin * Dv + tid; e < end * Dv; e += 256) {
      const int h = e / Dv, d = e - h * Dv;
      T* to = value_pages + (((size_t)page * kv_heads + h) * value_row + d) * block_size + slot;
      if (v_bias) store_from_float(to, biased(vrow, v_bias, e));
      else *to = vrow[e];
    }
  };
  if (gridDim.y == 1) {
    q_range(0, q_heads);
    if (page >= 0) {
      k_range(0, kv_heads);
      v_range(0, kv_heads);
    }
    return;
  }
  for (int unit = blockIdx.y; unit < units; unit += gridDim.y) {
    if (unit < q_heads) {
      q_range(unit, unit + 1);
    } else if (page >= 0 && unit < q_heads + kv_heads) {
      k_range(unit - q_heads, unit - q_heads + 1);
    } else if (page >= 0) {
      v_range(unit - q_heads - kv_heads, unit - q_heads - kv_heads + 1);
    }
  }
}

// The same in pieces of eight elements (16 bytes of bfloat16) where the sizes are multiples of eight.  The first
// tokens * parts blocks prepare q and k: a block reads its token's q and k once, adds the bias, keeps them in LDS as
// float32 and forms both sums of squares in one meeting; then it writes all heads (parts 1) or, in a step of few
// tokens, one (parts: q heads and k heads).  The blocks behind them write v: eight tokens times 256 dims a block, so that
// the eight slots of a dim, which lie together in the transposed pages, go out in one store where the tokens are
// eight neighbours that begin at a multiple of eight.
__device__ __forceinline__ void load8(const float* p, float v[8]) {
  const float4 a = ((const float4*)p)[0], b = ((const float4*)p)[1];
  v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
}
__device__ __forceinline__ void load8(const bf16_t* p, float v[8]) {
  const uint4 a = *(const uint4*)p;
  const uint32_t w[4] = {a.x, a.y, a.z, a.w};
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    v[2 * k] = __uint_as_float(w[k] << 16);
    v[2 * k + 1] = __uint_as_float(w[k] & 0xffff0000u);
  }
}
__device__ __forceinline__ void store8(float* p, const float v[8]) {
  ((float4*)p)[0] = make_float4(v[0], v[1], v[2], v[3]);
  ((float4*)p)[1] = make_float4(v[4], v[5], v[6], v[7]);
}
__device__ __forceinline__ void store8(bf16_t* p, const float v[8]) {
  uint32_t w[4];
#pragma unroll
  for (int k = 0; k < 4; ++k) w[k] = (uint32_t)float_to_bf16(v[2 * k]) | ((uint32_t)float_to_bf16(v[2 * k + 1]) << 16);
  *(uint4*)p = make_uint4(w[0], w[1], w[2], w[3]);
}

#define V_TOKENS 8

template <typename T>
__global__ __launch_bounds__(256) void whole_norm_rope_x8_kernel(
    const T* __restrict__ qkv, size_t stride, const float* __restrict__ bias, const float* __restrict__ q_weight,
    const float* __restrict__ k_weight, const float* __restrict__ inv_freq, const int* __restrict__ positions,
    const int* __restrict__ token_seq, const int* __restrict__ block_table, int table_stride, T* __restrict__ key_pages,
    T* __restrict__ value_pages, T* __restrict__ q_out, int tokens, int q_heads, int kv_heads, int D, int Dv, int R, float eps,
    float magnitude, int write_kv, int block_size, int num_blocks, int key_row, int value_row, int parts) {
  extern __shared__ __attribute__((aligned(16))) float held[];       // q, then k, biased
  __shared__ float cs[128], sn[128], sums[2][4];
  const int tid = threadIdx.x;
  const int q_size = q_heads * D, kv_size = kv_heads * D;
  const int qk_blocks = tokens * parts;

  if ((int)blockIdx.x >= qk_blocks) {
    const int width = kv_heads * Dv;
    const int across = (width + 255) / 256;
    const int b = blockIdx.x - qk_blocks;
    const int t0 = b / across * V_TOKENS, e = (b % across) * 256 + tid;
    if (e >= width) return;
    const int count = min(V_TOKENS, tokens - t0);
    const float shift = bias ? bias[q_size + kv_size + e] : 0.f;
    float v[V_TOKENS];
#pragma unroll
    for (int i = 0; i < V_TOKENS; ++i)
      v[i] = i < count ? load_as_float(qkv + (size_t)(t0 + i) * stride + q_size + kv_size + e) + shift : 0.f;
    const int h = e / Dv, d = e - h * Dv;
    auto page_of = [&](int t, int pos) {
      const int page = block_table[(size_t)token_seq[t] * table_stride + pos / block_size];
      return page < 0 || page >= num_blocks ? -1 : page;
    };
    auto at = [&](int page, int pos) { return value_pages + (((size_t)page * kv_heads + h) * value_row + d) * block_size + pos % block_size; };
    const int first = positions[t0];
    bool together = count == V_TOKENS && first % V_TOKENS == 0 && block_size % V_TOKENS == 0;
    if (together) together = positions[t0 + V_TOKENS - 1] == first + V_TOKENS - 1 && token_seq[t0 + V_TOKENS - 1] == token_seq[t0];
    if (together) {
      const int page = page_of(t0, first);
      if (page >= 0) store8(at(page, first), v);
      return;
    }
    for (int i = 0; i < count; ++i) {
      const int pos = positions[t0 + i], page = page_of(t0 + i, pos);
      if (page >= 0) store_from_float(at(page, pos), v[i]);
    }
    return;
  }

  const int t = blockIdx.x / parts, part = blockIdx.x % parts;
  const int pos = positions[t];
  const int half = R / 2;
  for (int j = tid; j < half; j += 256) {
    float s, c;
    sincosf((float)pos * inv_freq[j], &s, &c);
    cs[j] = c * magnitude;
    sn[j] = s * magnitude;
  }
  const T* row = qkv + (size_t)t * stride;
  const int q_pieces = q_size / 8, pieces = (q_size + (write_kv ? kv_size : 0)) / 8;
  float sq = 0.f, sk = 0.f;
  for (int p = tid; p < pieces; p += 256) {
    float v[8];
    load8(row + p * 8, v);
    if (bias) {
      float b[8];
      load8(bias + p * 8, b);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] += b[i];
    }
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) s = fmaf(v[i], v[i], s);
    if (p < q_pieces) sq += s;
    else sk += s;
    store8(held + p * 8, v);
  }
  sq = wave_sum_dpp(sq);
  sk = wave_sum_dpp(sk);
  if ((tid & 63) == 0) {
    sums[0][tid >> 6] = sq;
    sums[1][tid >> 6] = sk;
  }
  __syncthreads();
  const float inv_q = 1.f / sqrtf((sums[0][0] + sums[0][1] + sums[0][2] + sums[0][3]) / (float)q_size + eps);
  const float inv_k = 1.f / sqrtf((sums[1][0] + sums[1][1] + sums[1][2] + sums[1][3]) / (float)kv_size + eps);

  // piece d .. d + 7 of a head that begins at `at`, normed and turned
  auto turned = [&](const float* at, const float* w, float inv, int d, float v[8]) {
    float g[8];
    load8(at + d, v);
    load8(w + d, g);
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] *= inv * g[i];
    if (d >= R) return;
    const bool low = d < half;
    const int other = low ? d + half : d - half, j = low ? d : d - half;
    float o[8];
    load8(at + other, o);
    load8(w + other, g);
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const float partner = o[i] * inv * g[i];
      v[i] = low ? v[i] * cs[j + i] - partner * sn[j + i] : v[i] * cs[j + i] + partner * sn[j + i];
    }
  };
  int page = -1, slot = 0;
  if (write_kv) {
    page = block_table[(size_t)token_seq[t] * table_stride + pos / block_size];
    if (page < 0 || page >= num_blocks) page = -1;
    slot = pos % block_size;
  }
  const int heads = q_heads + (write_kv ? kv_heads : 0), per_head = key_row / 8;
  const int begin = parts == 1 ? 0 : part * per_head, end = parts == 1 ? heads * per_head : begin + per_head;
  for (int f = begin + tid; f < end; f += 256) {
    const int h = f / per_head, d = (f - h * per_head) * 8;
    const bool is_q = h < q_heads;
    const int hk = h - q_heads;
    if (!is_q && page < 0) continue;
    float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (d < D) {
      if (is_q) turned(held + h * D, q_weight + h * D, inv_q, d, v);
      else turned(held + q_size + hk * D, k_weight + hk * D, inv_k, d, v);
    }
    T* to = is_q ? q_out + ((size_t)t * q_heads + h) * key_row + d
                 : key_pages + (((size_t)page * kv_heads + hk) * block_size + slot) * key_row + d;
    store8(to, v);
  }
}

#define FEW_TOKENS 64                    // up to here a block writes one head
#define HELD_MAX_BYTES (48 * 1024)

extern "C" int fe_whole_norm_rope_write(const void* qkv, int dtype, long long stride, const float* bias, const float* q_weight,
                                        const float* k_weight, const float* inv_freq, const int* positions,
                                        const int* token_seq, const int* block_table, int table_stride, void* key_pages,
                                        void* value_pages, void* q_out, int tokens, int q_heads, int kv_heads,
                                        int head_dim, int value_dim, int rotary_dim, float eps, float magnitude,
                                        int write_kv, int block_size, int num_blocks, int key_row, int value_row,
                                        hipStream_t stream) {
  if (tokens <= 0) return FE_OK;
  const long long need = (long long)q_heads * head_dim + (write_kv ? (long long)kv_heads * (head_dim + value_dim) : 0);
  if (q_heads <= 0 || kv_heads <= 0 || head_dim <= 0 || value_dim <= 0 || rotary_dim < 0 || rotary_dim % 2 ||
      rotary_dim > head_dim || rotary_dim > 256 || stride < need || key_row < head_dim || value_row < value_dim || !(eps > 0.f) || !q_weight || (rotary_dim && !inv_freq) ||
      (write_kv && (!k_weight || !key_pages || !value_pages || !block_table || block_size <= 0 || num_blocks <= 0)))
    return FE_BAD_ARGUMENT;
  const size_t held = ((size_t)q_heads + (write_kv ? kv_heads : 0)) * head_dim * sizeof(float);
  const uintptr_t addresses = (uintptr_t)qkv | (uintptr_t)bias | (uintptr_t)q_weight | (uintptr_t)k_weight | (uintptr_t)key_pages |
                              (uintptr_t)value_pages | (uintptr_t)q_out;
  if (head_dim % 8 == 0 && rotary_dim % 16 == 0 && key_row % 8 == 0 && stride % 8 == 0 && (addresses & 15) == 0 && held <= HELD_MAX_BYTES) {
    const int parts = tokens <= FEW_TOKENS ? q_heads + (write_kv ? kv_heads : 0) : 1;
    const long long v_blocks = write_kv ? (long long)((tokens + V_TOKENS - 1) / V_TOKENS) * ((kv_heads * value_dim + 255) / 256) : 0;
    const long long blocks = (long long)tokens * parts + v_blocks;
    if (blocks > 0x7fffffffLL) return FE_BAD_ARGUMENT;
#define LAUNCH8(T)                                                                                                     \
  whole_norm_rope_x8_kernel<T><<<(unsigned)blocks, 256, held, stream>>>(                                               \
      (const T*)qkv, (size_t)stride, bias, q_weight, k_weight, inv_freq, positions, token_seq, block_table, table_stride, \
      (T*)key_pages, (T*)value_pages, (T*)q_out, tokens, q_heads, kv_heads, head_dim, value_dim, rotary_dim, eps, magnitude, \
      write_kv, block_size, num_blocks, key_row, value_row, parts)
    if (dtype == FE_F32) LAUNCH8(float);
    else if (dtype == FE_BF16) LAUNCH8(bf16_t);
    else return FE_BAD_ARGUMENT;
#undef LAUNCH8
    return fe_check_launch();
  }
  const int units = q_heads + (write_kv ? 2 * kv_heads : 0);
  const dim3 grid(tokens, tokens <= 256 ? (units < 65535 ? units : 65535) : 1);
#define LAUNCH(T)                                                                                                      \
  whole_norm_rope_kernel<T><<<grid, 256, 0, stream>>>((const T*)qkv, (size_t)stride, bias, q_weight, k_weight, inv_freq,   \
                                                        positions, token_seq, block_table, table_stride, (T*)key_pages, \
                                                        (T*)value_pages, (T*)q_out, q_heads, kv_heads, head_dim,       \
                                                        value_dim, rotary_dim, eps, magnitude, write_kv, block_size,   \
                                                        num_blocks, key_row, value_row)
  if (dtype == FE_F32) LAUNCH(float);
  else if (dtype == FE_BF16) LAUNCH(bf16_t);
  else return FE_BAD_ARGUMENT;
#undef LAUNCH
  return fe_check_launch();
}
