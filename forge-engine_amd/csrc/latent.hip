// Attention through a latent: what lies between its products.
//
//   fe_latent_norm_rope_write: from the fused down-projections of a token, x = [a | b | r] (float32 or the cache's
//       dtype: a of q_rank, b of kv_rank, r of rot_dim entries), the query latent a / rms(a) * wq into cq [T, q_rank]
//       (q_rank 0: none) and, for a layer that caches, the token's cache row [b / rms(b) * wkv | 0 | rotate(r) | 0] into its
//       page (key pages [page][1][slot][key_row]: the latent part is value_row wide, the rotated part the rest; both
//       are filled up with zeros where the pages are wider than what they hold) and, where the cache keeps values, the
//       normed b a second time into the transposed value pages ([page][1][value_row][slot], the layout the matrix-core
//       attention reads its second operand in; dims beyond kv_rank are left alone).  The rotation turns the first
//       rotary_dim dims of r by the angle position * inv_freq[i], cosines and sines times `magnitude`: dim i with
//       dim i + rotary_dim / 2, or (interleaved) dim 2i with dim 2i + 1; the rest pass.
//   fe_latent_query_pack: the attention's query rows [T, heads, key_row], laid out like a cache row, from the queries
//       taken through the key up-projection (qa [heads, T, value_row], the result of a batched product) and
//       the rotated part of every head of q [T, heads, dim + rot_dim], rotated here.
//   fe_latent_gate_heads: the heads' results x [heads, T, dim] (of a batched product) side by side, [T, heads * dim],
//       times sigmoid(gate) element by element if there is a gate.
//   fe_latent_query_step, fe_latent_value_step: a few tokens (up to 16, bfloat16): the product per head and what follows
//       it in one launch, the weight streamed once on the matrix cores: queries through the key up-projection straight into
//       the query rows (with the rotated parts), and the attention's results through the value up-projection, gated.
// Norms, angles, rotations and gates are float32, one rounding at the stores.
#include "common.h"

#define LT_THREADS 256

// Where pair i of a rotation lies.
struct Pairing {
  int step, offset;     // dims i * step and i * step + offset
};
static inline Pairing pairing(int rotary_dim, int interleaved) { return interleaved ? Pairing{2, 1} : Pairing{1, rotary_dim / 2}; }

template <typename TX, typename T>
__global__ __launch_bounds__(LT_THREADS) void latent_norm_rope_write_kernel(
    const TX* __restrict__ x, size_t stride, int q_rank, int kv_rank, int rot_dim, int rotary_dim,
    const float* __restrict__ wq, const float* __restrict__ wkv, const float* __restrict__ inv_freq,
    const int* __restrict__ positions, const int* __restrict__ token_seq, const int* __restrict__ block_table,
    int table_stride, T* __restrict__ key_pages, T* __restrict__ value_pages, T* __restrict__ cq, float eps,
    int block_size, int num_blocks, int write_kv, int key_row, int value_row, Pairing pairs, float magnitude) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, tid = threadIdx.x;
  const TX* row = x + (size_t)t * stride;
  if (q_rank) {
    float ss = 0.f;
    for (int c = tid; c < q_rank; c += LT_THREADS) {
      const float v = load_as_float(row + c);
      ss += v * v;
    }
    ss = block_sum<true>(ss, scratch);
    const float inv_q = rsqrtf(ss / (float)q_rank + eps);
    for (int c = tid; c < q_rank; c += LT_THREADS)
      store_from_float(cq + (size_t)t * q_rank + c, load_as_float(row + c) * inv_q * wq[c]);
  }
  if (!write_kv) return;

  const TX* b = row + q_rank;
  float sb = 0.f;
  for (int c = tid; c < kv_rank; c += LT_THREADS) {
    const float v = load_as_float(b + c);
    sb += v * v;
  }
  sb = block_sum(sb, scratch);
  const float inv_b = rsqrtf(sb / (float)kv_rank + eps);
  const int pos = positions[t];
  const int page = block_table[(size_t)token_seq[t] * table_stride + pos / block_size];
  if (page < 0 || page >= num_blocks) return;
  T* dst = key_pages + ((size_t)page * block_size + pos % block_size) * key_row;
  T* vdst = value_pages ? value_pages + (size_t)page * value_row * block_size + pos % block_size : nullptr;
  for (int c = tid; c < kv_rank; c += LT_THREADS) {
    const float v = load_as_float(b + c) * inv_b * wkv[c];
    store_from_float(dst + c, v);
    if (vdst) store_from_float(vdst + (size_t)c * block_size, v);
  }
  for (int c = kv_rank + tid; c < value_row; c += LT_THREADS) store_from_float(dst + c, 0.f);
  const TX* r = b + kv_rank;
  T* turned = dst + value_row;
  for (int i = tid; i < rotary_dim / 2; i += LT_THREADS) {
    float sn, cs;
    sincosf((float)pos * inv_freq[i], &sn, &cs);
    cs *= magnitude;
    sn *= magnitude;
    const int lo = i * pairs.step, hi = lo + pairs.offset;
    const float u = load_as_float(r + lo), v = load_as_float(r + hi);
    store_from_float(turned + lo, u * cs - v * sn);
    store_from_float(turned + hi, v * cs + u * sn);
  }
  for (int c = rotary_dim + tid; c < key_row - value_row; c += LT_THREADS)
    store_from_float(turned + c, c < rot_dim ? load_as_float(r + c) : 0.f);
}

extern "C" int fe_latent_norm_rope_write(const void* x, int x_dtype, long long stride, int q_rank, int kv_rank, int rot_dim,
                                         int rotary_dim, const float* wq, const float* wkv, const float* inv_freq,
                                         const int* positions, const int* token_seq, const int* block_table,
                                         int table_stride, void* key_pages, void* value_pages, void* cq, int dtype, float eps, int tokens,
                                         int block_size, int num_blocks, int write_kv, int key_row, int value_row,
                                         int interleaved, float magnitude, hipStream_t stream) {
  if (tokens <= 0) return FE_OK;
  if (q_rank < 0 || kv_rank < 1 || rot_dim < 0 || rotary_dim < 0 || rotary_dim > rot_dim || rotary_dim % 2 || !(eps > 0.f) ||
      !x || (q_rank && (!wq || !cq)) || (!q_rank && !write_kv))
    return FE_BAD_ARGUMENT;
  if (stride < (long long)q_rank + (write_kv ? kv_rank + rot_dim : 0)) return FE_BAD_ARGUMENT;
  if (write_kv && (!wkv || !key_pages || !positions || !token_seq || !block_table || block_size < 1 || num_blocks < 1 ||
                   (rotary_dim && !inv_freq) || value_row < kv_rank || key_row < value_row + rot_dim))
    return FE_BAD_ARGUMENT;
#define LAUNCH(TX, T)                                                                                                \
  latent_norm_rope_write_kernel<TX, T><<<tokens, LT_THREADS, 0, stream>>>(                                           \
      (const TX*)x, (size_t)stride, q_rank, kv_rank, rot_dim, rotary_dim, wq, wkv, inv_freq, positions, token_seq, block_table, \
      table_stride, (T*)key_pages, (T*)value_pages, (T*)cq, eps, block_size, num_blocks, write_kv, key_row, value_row,     \
      pairing(rotary_dim, interleaved), magnitude)
  if (x_dtype == FE_F32 && dtype == FE_F32) LAUNCH(float, float);
  else if (x_dtype == FE_F32 && dtype == FE_BF16) LAUNCH(float, bf16_t);
  else if (x_dtype == FE_BF16 && dtype == FE_BF16) LAUNCH(bf16_t, bf16_t);
  else return FE_BAD_ARGUMENT;
#undef LAUNCH
  return fe_check_launch();
}

// One wave per (token, head).
template <typename T>
__global__ __launch_bounds__(64) void latent_query_pack_kernel(
    const T* __restrict__ q, size_t q_stride, const T* __restrict__ qa, const float* __restrict__ inv_freq,
    const int* __restrict__ positions, T* __restrict__ out, int tokens, int heads, int dim, int rot_dim, int rotary_dim,
    int key_row, int value_row, Pairing pairs, float magnitude) {
  const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  T* dst = out + ((size_t)t * heads + h) * key_row;
  const T* a = qa + ((size_t)h * tokens + t) * value_row;
  constexpr int PER = 16 / sizeof(T);
  if (value_row % PER == 0 && key_row % PER == 0 && ((((uintptr_t)qa) | ((uintptr_t)out)) & 15) == 0) {
    for (int c = lane; c < value_row / PER; c += 64) ((uint4*)dst)[c] = ((const uint4*)a)[c];
  } else {
    for (int c = lane; c < value_row; c += 64) dst[c] = a[c];
  }
  const T* r = q + (size_t)t * q_stride + (size_t)h * (dim + rot_dim) + dim;
  T* turned = dst + value_row;
  const int pos = positions[t];
  for (int i = lane; i < rotary_dim / 2; i += 64) {
    float sn, cs;
    sincosf((float)pos * inv_freq[i], &sn, &cs);
    cs *= magnitude;
    sn *= magnitude;
    const int lo = i * pairs.step, hi = lo + pairs.offset;
    const float u = load_as_float(r + lo), v = load_as_float(r + hi);
    store_from_float(turned + lo, u * cs - v * sn);
    store_from_float(turned + hi, v * cs + u * sn);
  }
  for (int c = rotary_dim + lane; c < key_row - value_row; c += 64) {
    if (c < rot_dim) turned[c] = r[c];
    else store_from_float(turned + c, 0.f);
  }
}

extern "C" int fe_latent_query_pack(const void* q, long long q_stride, const void* qa, const float* inv_freq,
                                    const int* positions, void* out, int dtype, int tokens, int heads, int dim,
                                    int rot_dim, int rotary_dim, int key_row, int value_row, int interleaved, float magnitude,
                                    hipStream_t stream) {
  if (tokens <= 0) return FE_OK;
  if (heads < 1 || heads > 65535 || dim < 1 || value_row < 1 || rot_dim < 0 || rotary_dim < 0 || rotary_dim > rot_dim ||
      rotary_dim % 2 || q_stride < (long long)heads * (dim + rot_dim) || key_row < value_row + rot_dim || !q || !qa || !out ||
      !positions || (rotary_dim && !inv_freq))
    return FE_BAD_ARGUMENT;
  const dim3 grid(tokens, heads);
#define LAUNCH(T)                                                                                          \
  latent_query_pack_kernel<T><<<grid, 64, 0, stream>>>((const T*)q, (size_t)q_stride, (const T*)qa, inv_freq, \
                                                       positions, (T*)out, tokens, heads, dim, rot_dim, rotary_dim, key_row, \
                                                       value_row, pairing(rotary_dim, interleaved), magnitude)
  if (dtype == FE_F32) LAUNCH(float);
  else if (dtype == FE_BF16) LAUNCH(bf16_t);
  else return FE_BAD_ARGUMENT;
#undef LAUNCH
  return fe_check_launch();
}

// ---------------------------------------------------------------- a few tokens: product per head with its ending
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) float floatx4;
typedef __attribute__((ext_vector_type(4))) unsigned int uintx4;

#define STEP_TOKENS 16

// y[t][n] = sum_k x[t][k] w[n][k] for one head, 16 columns n from n0 on; w [N, K] with K contiguous, a multiple of 8.
// Block = 4 waves that share K in steps of 32; thread (m, c) = (tid / 16, tid % 16) returns y[m][n0 + c].
__device__ __forceinline__ float head_tile(const bf16_t* __restrict__ x, size_t token_stride, const bf16_t* __restrict__ w,
                                           int tokens, int N, int K, int n0, float (*red)[64][4]) {
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lr = lane & 15, lq = lane >> 4;
  const bool row_ok = lr < tokens, col_ok = n0 + lr < N;
  const bf16_t* xrow = x + (size_t)(row_ok ? lr : 0) * token_stride + lq * 8;
  const bf16_t* wrow = w + (size_t)(col_ok ? n0 + lr : 0) * K + lq * 8;
  const uintx4 none = uintx4{0u, 0u, 0u, 0u};
  floatx4 acc = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int k = wave * 32; k < K; k += 128) {
    const bool in = k + lq * 8 < K;
    const uintx4 a = in && row_ok ? *(const uintx4*)(xrow + k) : none;
    const uintx4 b = in && col_ok ? *(const uintx4*)(wrow + k) : none;
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), acc, 0, 0, 0);
  }
  *(floatx4*)red[wave][lane] = acc;        // lane (lr, lq): rows 4 lq + i of column lr
  __syncthreads();
  const int m = tid >> 4, c = tid & 15;
  float y = 0.f;
#pragma unroll
  for (int wv = 0; wv < 4; ++wv) y += red[wv][(m >> 2) * 16 + c][m & 3];
  return y;
}

// Blocks (column tile, head); the last column tile's index stands for the head's rotated parts instead.
__global__ __launch_bounds__(256) void latent_query_step_kernel(
    const bf16_t* __restrict__ q, size_t q_stride, const bf16_t* __restrict__ uk, const float* __restrict__ inv_freq,
    const int* __restrict__ positions, bf16_t* __restrict__ out, int tokens, int heads, int dim, int rot_dim, int rotary_dim,
    int key_row, int value_row, Pairing pairs, float magnitude) {
  __shared__ __attribute__((aligned(16))) float red[4][64][4];
  const int h = blockIdx.y, tid = threadIdx.x;
  const bf16_t* x = q + (size_t)h * (dim + rot_dim);
  if (blockIdx.x + 1 < gridDim.x) {
    const int n0 = blockIdx.x * 16;
    const float y = head_tile(x, q_stride, uk + (size_t)h * value_row * dim, tokens, value_row, dim, n0, red);
    const int m = tid >> 4, n = n0 + (tid & 15);
    if (m < tokens && n < value_row) out[((size_t)m * heads + h) * key_row + n] = float_to_bf16(y);
    return;
  }
  const int half = rotary_dim / 2;
  for (int e = tid; e < tokens * half; e += 256) {
    const int t = e / half, i = e - t * half;
    float sn, cs;
    sincosf((float)positions[t] * inv_freq[i], &sn, &cs);
    cs *= magnitude;
    sn *= magnitude;
    const bf16_t* r = x + (size_t)t * q_stride + dim;
    bf16_t* turned = out + ((size_t)t * heads + h) * key_row + value_row;
    const int lo = i * pairs.step, hi = lo + pairs.offset;
    const float u = bf16_to_float(r[lo]), v = bf16_to_float(r[hi]);
    turned[lo] = float_to_bf16(u * cs - v * sn);
    turned[hi] = float_to_bf16(v * cs + u * sn);
  }
  const int rest = key_row - value_row - rotary_dim;
  for (int e = tid; e < tokens * rest; e += 256) {
    const int t = e / rest, c = rotary_dim + e - t * rest;
    out[((size_t)t * heads + h) * key_row + value_row + c] = c < rot_dim ? x[(size_t)t * q_stride + dim + c] : (bf16_t)0;
  }
}

extern "C" int fe_latent_query_step(const void* q, long long q_stride, const void* uk, const float* inv_freq, const int* positions,
                                    void* out, int tokens, int heads, int dim, int rot_dim, int rotary_dim, int key_row,
                                    int value_row, int interleaved, float magnitude, hipStream_t stream) {
  if (tokens <= 0) return FE_OK;
  if (tokens > STEP_TOKENS || heads < 1 || heads > 65535 || dim < 8 || dim % 8 || (dim + rot_dim) % 8 || q_stride % 8 || value_row < 1 ||
      rot_dim < 0 || rotary_dim < 0 || rotary_dim > rot_dim || rotary_dim % 2 || q_stride < (long long)heads * (dim + rot_dim) ||
      key_row < value_row + rot_dim || !q || !uk || !out || !positions || (rotary_dim && !inv_freq) ||
      ((((uintptr_t)q) | ((uintptr_t)uk)) & 15))
    return FE_BAD_ARGUMENT;
  latent_query_step_kernel<<<dim3((value_row + 15) / 16 + 1, heads), 256, 0, stream>>>(
      (const bf16_t*)q, (size_t)q_stride, (const bf16_t*)uk, inv_freq, positions, (bf16_t*)out, tokens, heads, dim, rot_dim, rotary_dim,
      key_row, value_row, pairing(rotary_dim, interleaved), magnitude);
  return fe_check_launch();
}

__global__ __launch_bounds__(256) void latent_value_step_kernel(const bf16_t* __restrict__ x, const bf16_t* __restrict__ uv,
                                                                const bf16_t* __restrict__ gate, size_t gate_stride,
                                                                bf16_t* __restrict__ out, int tokens, int heads, int latent, int dim) {
  __shared__ __attribute__((aligned(16))) float red[4][64][4];
  const int h = blockIdx.y, n0 = blockIdx.x * 16, m = threadIdx.x >> 4, n = n0 + (threadIdx.x & 15);
  const bool mine = m < tokens && n < dim;
  const float g = mine && gate ? bf16_to_float(gate[(size_t)m * gate_stride + (size_t)h * dim + n]) : 0.f;
  const float y = head_tile(x + (size_t)h * latent, (size_t)heads * latent, uv + (size_t)h * dim * latent, tokens, dim, latent, n0, red);
  if (mine) out[(size_t)m * heads * dim + (size_t)h * dim + n] = float_to_bf16(gate ? y / (1.f + expf(-g)) : y);
}

extern "C" int fe_latent_value_step(const void* x, const void* uv, const void* gate, long long gate_stride, void* out, int tokens,
                                    int heads, int latent, int dim, hipStream_t stream) {
  if (tokens <= 0) return FE_OK;
  if (tokens > STEP_TOKENS || heads < 1 || heads > 65535 || latent < 8 || latent % 8 || dim < 1 || !x || !uv || !out ||
      (gate && gate_stride < (long long)heads * dim) || ((((uintptr_t)x) | ((uintptr_t)uv)) & 15))
    return FE_BAD_ARGUMENT;
  latent_value_step_kernel<<<dim3((dim + 15) / 16, heads), 256, 0, stream>>>((const bf16_t*)x, (const bf16_t*)uv, (const bf16_t*)gate,
                                                                           (size_t)gate_stride, (bf16_t*)out, tokens, heads, latent, dim);
  return fe_check_launch();
}

template <typename T>
__device__ __forceinline__ float gated(float v, const T* gate) { return gate ? v / (1.f + expf(-load_as_float(gate))) : v; }

template <typename T>
__global__ __launch_bounds__(256) void latent_gate_heads_kernel(const T* __restrict__ x, const T* __restrict__ gate,
                                                                size_t gate_stride, T* __restrict__ out, int tokens, int heads,
                                                                int dim, long long count) {
  const long long i = (long long)blockIdx.x * 256 + threadIdx.x;
  if (i >= count) return;
  const int width = heads * dim;
  const int t = (int)(i / width), c = (int)(i - (long long)t * width);
  const int h = c / dim, d = c - h * dim;
  const float v = load_as_float(x + ((size_t)h * tokens + t) * dim + d);
  store_from_float(out + i, gated(v, gate ? gate + (size_t)t * gate_stride + c : nullptr));
}

// bfloat16 in pieces of 16 bytes
__global__ __launch_bounds__(256) void latent_gate_heads_bf16x8_kernel(const bf16_t* __restrict__ x, const bf16_t* __restrict__ gate,
                                                                       size_t gate_stride, bf16_t* __restrict__ out, int tokens,
                                                                       int heads, int dim8, long long count8) {
  const long long i = (long long)blockIdx.x * 256 + threadIdx.x;
  if (i >= count8) return;
  const int width8 = heads * dim8;
  const int t = (int)(i / width8), c = (int)(i - (long long)t * width8);
  const int h = c / dim8, d = c - h * dim8;
  uint4 v = ((const uint4*)x)[((size_t)h * tokens + t) * dim8 + d];
  if (gate) {
    const uint4 g = *(const uint4*)(gate + (size_t)t * gate_stride + (size_t)c * 8);
    const uint32_t vw[4] = {v.x, v.y, v.z, v.w}, gw[4] = {g.x, g.y, g.z, g.w};
    uint32_t ow[4];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const float lo = __uint_as_float(vw[k] << 16) / (1.f + expf(-__uint_as_float(gw[k] << 16)));
      const float hi = __uint_as_float(vw[k] & 0xffff0000u) / (1.f + expf(-__uint_as_float(gw[k] & 0xffff0000u)));
      ow[k] = (uint32_t)float_to_bf16(lo) | ((uint32_t)float_to_bf16(hi) << 16);
    }
    v = make_uint4(ow[0], ow[1], ow[2], ow[3]);
  }
  ((uint4*)out)[i] = v;
}

extern "C" int fe_latent_gate_heads(const void* x, const void* gate, long long gate_stride, void* out, int dtype, int tokens,
                                    int heads, int dim, hipStream_t stream) {
  if (tokens <= 0) return FE_OK;
  if (heads < 1 || dim < 1 || !x || !out || (gate && gate_stride < (long long)heads * dim)) return FE_BAD_ARGUMENT;
  const long long count = (long long)tokens * heads * dim;
  if (count / 256 >= 0x7fffffffLL) return FE_BAD_ARGUMENT;
  if (dtype == FE_BF16 && dim % 8 == 0 && gate_stride % 8 == 0 && ((((uintptr_t)x) | ((uintptr_t)gate) | ((uintptr_t)out)) & 15) == 0) {
    latent_gate_heads_bf16x8_kernel<<<(int)((count / 8 + 255) / 256), 256, 0, stream>>>(
        (const bf16_t*)x, (const bf16_t*)gate, (size_t)gate_stride, (bf16_t*)out, tokens, heads, dim / 8, count / 8);
    return fe_check_launch();
  }
  const int blocks = (int)((count + 255) / 256);
  if (dtype == FE_F32)
    latent_gate_heads_kernel<float><<<blocks, 256, 0, stream>>>((const float*)x, (const float*)gate, (size_t)gate_stride, (float*)out,
                                                                tokens, heads, dim, count);
  else if (dtype == FE_BF16)
    latent_gate_heads_kernel<bf16_t><<<blocks, 256, 0, stream>>>((const bf16_t*)x, (const bf16_t*)gate, (size_t)gate_stride,
                                                                 (bf16_t*)out, tokens, heads, dim, count);
  else return FE_BAD_ARGUMENT;
  return fe_check_launch();
}
