// Linear recurrences over a matrix state whose decay is one number per head and token (retention, the
// state-space duality of Mamba-2), over a mixed batch:
//     S_t = exp(l_t) S_(t-1) + b_t k_t v_t^T,      o_t = S_t^T q_t (+ skip_h v_t)
// l_t: a constant per head, or rate_h * dt_t with the step size dt_t = softplus(x_t + bias_h), which is
// then b_t as well.  q and k may be turned by a table of cosines and sines (dim i pairs with i + half), k may be
// scaled, and several heads may share one head of q and k.  S lives in the sequence's state slot [slots][heads]
// [value dim][key dim] (float32, value-major), is read at a step's start and written at its end: a sequence may be
// cut into steps anywhere.
//
// Prompts (fe_head_recurrence): chunks of 32 tokens as products on the matrix cores with 32-bit operands
// (v_mfma_f32_16x16x4_f32: everything that enters the recurrence stays float32).  With L_i the sum of l over the
// chunk's tokens up to i:
//     O_i  = exp(L_i) S^T q_i + sum_{j <= i} (q_i . k_j) exp(L_i - L_j) b_j v_j
//     S   <- exp(L_end) S + sum_j exp(L_end - L_j) b_j k_j v_j^T
// every exponent is a difference within one chunk and never positive where decays are at most one; the sums L are
// kept in 64-bit, so that a large step ahead of small ones does not eat their digits.
// Block = 4 waves on one head's chunk and 64 value columns, a wave owning 16 columns.  The state is the MFMA's
// accumulator: tile t of a wave holds S[16 t + 4 (lane / 16) + r][lane % 16], which is also exactly the operand
// that the product q S wants if a lane group takes key dims 4 (lane / 16) + m in step m (a product's inner index
// may be permuted freely as long as both operands agree), so the state never leaves its registers.  The same
// permutation lets every row-major operand be read as 16-byte pieces, and the values come from memory straight
// into the operand's place.  Scores q k^T of the chunk are formed once by three waves (the lower triangle of
// 2 x 2 tiles) and meet the other waves through LDS.
// A long sequence is cut into segments walked side by side: a first launch (SUMMARY) walks every segment but a
// sequence's last from a zero state without read-outs, head_combine_kernel chains the segments' end states into
// the states ahead of them, a second launch walks every segment from its true start.  A sequence's segments are found from the lengths on the
// device, so captured steps are laid out for the token count alone.
//
// Single tokens (fe_head_recurrence_step): block = one head of one sequence, 16 lanes share a column of the
// state, which is read and written once; with a gate the head's read-out is divided by its root mean square and
// multiplied by silu(gate) in the same launch.
#include "common.h"

#define HR_CHUNK 32
#define HR_COLS 64
#define HR_THREADS 256
#define HR_LOG2E 1.4426950408889634074

typedef __attribute__((ext_vector_type(4))) float floatx4;

struct HeadRecurrenceArgs {
  const void* q; const void* k; const void* v; const void* dt;
  size_t q_stride, k_stride, v_stride, dt_stride;
  const float* table;                // [tokens][rotary_dim / 2][2]: cosine, sine
  const float* rate;                 // [heads]: l per token, or its factor on dt
  const float* dt_bias; const float* skip;
  float* state; float* out;
  float* seg_state; double* seg_sum;
  const int* cu_q; const int* state_slots;
  float q_scale, k_scale;
  int rotary_dim, heads, share, key_dim, value_dim, tokens, num_seqs, slots, seg_len, column_blocks;
};

__device__ __forceinline__ float hr_softplus(float v) { return v > 20.f ? v : log1pf(expf(v)); }
__device__ __forceinline__ float hr_silu(float v) { return v / (1.f + expf(-v)); }

template <typename T> struct alignas(sizeof(T) * 4) Quad { T e[4]; };

// The sequence and segment behind a slot: sequence s's segments have the slots cu_q[s] / seg_len + s and up (runs
// of slots do not overlap: a sequence of n tokens has at most n / seg_len + 1 segments).  Every lane looks at some of
// the sequences, so that finding the slot takes one trip to memory.
__device__ __forceinline__ bool find_segment(const HeadRecurrenceArgs& p, int slot, int& seq, int& begin, int& end, bool& last) {
  const int lane = threadIdx.x & 63;
  int below = 0;
  for (int s0 = 0; s0 < p.num_seqs; s0 += 64) {
    const int s = s0 + lane;
    const bool before = s < p.num_seqs && p.cu_q[min(s, p.num_seqs - 1)] / p.seg_len + s <= slot;
    below += __popcll(__ballot(before));
  }
  seq = below - 1;
  if (seq < 0) return false;
  const int seq_begin = p.cu_q[seq], seq_end = p.cu_q[seq + 1];
  const int index = slot - (seq_begin / p.seg_len + seq);
  begin = seq_begin + index * p.seg_len;
  if (seq_end > p.tokens || begin >= seq_end) return false;
  end = min(seq_end, begin + p.seg_len);
  last = end == seq_end;
  return true;
}

// NT: tiles of 16 key dims; VEC: 4 neighbouring dims a load (the caller has checked sizes and alignment) or 1.
template <typename T, int NT, int VEC, bool ROT, bool SUMMARY>
__global__ __launch_bounds__(HR_THREADS) void head_recurrence_kernel(HeadRecurrenceArgs p) {
  constexpr int DKP = 16 * NT, ROW = DKP + 4, C = HR_CHUNK;
  constexpr int GROUPS = DKP / (2 * VEC);                                     // a group: VEC dims and their VEC partners
  constexpr int ITEMS = (C * GROUPS + HR_THREADS - 1) / HR_THREADS;           // groups of a chunk a thread stages
  __shared__ __attribute__((aligned(16))) float Qs[SUMMARY ? 1 : C][ROW];
  __shared__ __attribute__((aligned(16))) float Ks[C][ROW];
  __shared__ __attribute__((aligned(16))) float Ps[SUMMARY ? 1 : C][C + 4];
  __shared__ __attribute__((aligned(16))) float grow[C], weigh[C], scale_in[C];   // exp(L_i), exp(L_end - L_j) b_j, b_j
  __shared__ double sums[C];                                                      // L_i log2 e

  int seq, begin, end;
  bool last;
  const int slot_index = blockIdx.y;
  if (!find_segment(p, slot_index, seq, begin, end, last)) return;
  if (SUMMARY && last) return;
  const int slot = p.state_slots[seq];
  if (slot < 0 || slot >= p.slots) return;
  const int h = blockIdx.x / p.column_blocks, column0 = (blockIdx.x % p.column_blocks) * HR_COLS;
  const int tid = threadIdx.x, wave = tid / 64, lane = tid % 64, lr = lane % 16, lq = lane / 16;
  const int Dk = p.key_dim, Dv = p.value_dim, H = p.heads;
  const int column = column0 + wave * 16 + lr;
  const bool live_column = column < Dv;
  const int column_at = min(column, Dv - 1);
  const size_t head_at = (size_t)(h / p.share) * Dk;
  const double rate = (double)p.rate[h] * HR_LOG2E;
  const float skip = p.skip ? p.skip[h] : 0.f;
  const int half = ROT ? p.rotary_dim / 2 : 0;

  // the state: from the slot (a sequence in one segment), from where the combination left it, or zero
  floatx4 S[NT];
  float* home = p.state + (((size_t)slot * H + h) * Dv + column_at) * Dk;
  const bool whole_step = last && begin == p.cu_q[seq];
  {
    const float* from = whole_step ? home : p.seg_state + (((size_t)slot_index * H + h) * Dv + column_at) * Dk;
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = t * 16 + lq * 4 + r;
        S[t][r] = (!SUMMARY && live_column && d < Dk) ? from[d] : 0.f;
      }
  }
  // key dims beyond the real ones stay zero
  for (int e = tid; e < C * (DKP - Dk); e += HR_THREADS) {
    const int row = e / (DKP - Dk), d = Dk + e % (DKP - Dk);
    Ks[row][d] = 0.f;
    if (!SUMMARY) Qs[row][d] = 0.f;
  }

  // a group's first dim and its partners': turned pairs first, then what passes unchanged
  auto group_dims = [&](int u, int& lo, int& hi) {
    lo = u * VEC < half ? u * VEC : 2 * half + (u * VEC - half) * 2;
    hi = u * VEC < half ? lo + half : lo + VEC;
  };
  struct Item { Quad<T> q[2], k[2]; float4 turn[2]; };
  Item items[VEC == 4 ? ITEMS : 1];
  T v_raw[8];
  float dt_raw = 0.f;
  auto fetch = [&](int t0) {
    if constexpr (VEC == 4) {
#pragma unroll
      for (int n = 0; n < ITEMS; ++n) {
        const int e = min(tid + n * HR_THREADS, C * GROUPS - 1);
        const int row = e / GROUPS, u = min(e % GROUPS, Dk / (2 * VEC) - 1);
        const size_t t = (size_t)min(t0 + row, end - 1);
        int lo, hi;
        group_dims(u, lo, hi);
        const T* k = (const T*)p.k + t * p.k_stride + head_at;
        items[n].k[0] = *(const Quad<T>*)(k + lo);
        items[n].k[1] = *(const Quad<T>*)(k + hi);
        if constexpr (!SUMMARY) {
          const T* q = (const T*)p.q + t * p.q_stride + head_at;
          items[n].q[0] = *(const Quad<T>*)(q + lo);
          items[n].q[1] = *(const Quad<T>*)(q + hi);
        }
        if constexpr (ROT) {
          const float4* turn = (const float4*)(p.table + (t * half + min(lo, half - VEC)) * 2);
          items[n].turn[0] = turn[0];
          items[n].turn[1] = turn[1];
        }
      }
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const size_t t = (size_t)min(t0 + (i / 4) * 16 + lq * 4 + i % 4, end - 1);
      v_raw[i] = ((const T*)p.v)[t * p.v_stride + (size_t)h * Dv + column_at];
    }
    if (p.dt && wave == 0) dt_raw = load_as_float((const T*)p.dt + (size_t)min(t0 + lane, end - 1) * p.dt_stride + h);
  };
  auto turn_pair = [&](float& a, float& b, float cs, float sn) {
    const float u = a, w = b;
    a = u * cs - w * sn;
    b = w * cs + u * sn;
  };
  auto stage = [&](int t0) {
    if constexpr (VEC == 4) {
#pragma unroll
      for (int n = 0; n < ITEMS; ++n) {
        const int e = tid + n * HR_THREADS;
        const int row = e / GROUPS, u = e % GROUPS;
        if (e >= C * GROUPS || u >= Dk / (2 * VEC)) continue;
        int lo, hi;
        group_dims(u, lo, hi);
        const float live = t0 + row < end ? 1.f : 0.f;
        float k[2][4], q[2][4];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          k[0][i] = load_as_float(&items[n].k[0].e[i]);
          k[1][i] = load_as_float(&items[n].k[1].e[i]);
          if constexpr (!SUMMARY) {
            q[0][i] = load_as_float(&items[n].q[0].e[i]);
            q[1][i] = load_as_float(&items[n].q[1].e[i]);
          }
        }
        if constexpr (ROT) {
          if (u * VEC < half) {
            const float turn[8] = {items[n].turn[0].x, items[n].turn[0].y, items[n].turn[0].z, items[n].turn[0].w,
                                   items[n].turn[1].x, items[n].turn[1].y, items[n].turn[1].z, items[n].turn[1].w};
#pragma unroll
            for (int i = 0; i < 4; ++i) {
              turn_pair(k[0][i], k[1][i], turn[2 * i], turn[2 * i + 1]);
              if constexpr (!SUMMARY) turn_pair(q[0][i], q[1][i], turn[2 * i], turn[2 * i + 1]);
            }
          }
        }
        const float ks = live * p.k_scale;
        *(float4*)&Ks[row][lo] = make_float4(k[0][0] * ks, k[0][1] * ks, k[0][2] * ks, k[0][3] * ks);
        *(float4*)&Ks[row][hi] = make_float4(k[1][0] * ks, k[1][1] * ks, k[1][2] * ks, k[1][3] * ks);
        if constexpr (!SUMMARY) {
          const float qs = live * p.q_scale;
          *(float4*)&Qs[row][lo] = make_float4(q[0][0] * qs, q[0][1] * qs, q[0][2] * qs, q[0][3] * qs);
          *(float4*)&Qs[row][hi] = make_float4(q[1][0] * qs, q[1][1] * qs, q[1][2] * qs, q[1][3] * qs);
        }
      }
    } else {
      for (int e = tid; e < C * GROUPS; e += HR_THREADS) {
        const int row = e / GROUPS, u = e % GROUPS;
        int lo, hi;
        group_dims(u, lo, hi);
        if (lo >= Dk) continue;
        const int partner = min(hi, Dk - 1);
        const size_t t = (size_t)min(t0 + row, end - 1);
        const float live = t0 + row < end ? 1.f : 0.f;
        const T* k = (const T*)p.k + t * p.k_stride + head_at;
        float k0 = load_as_float(k + lo), k1 = load_as_float(k + partner), q0 = 0.f, q1 = 0.f;
        if constexpr (!SUMMARY) {
          const T* q = (const T*)p.q + t * p.q_stride + head_at;
          q0 = load_as_float(q + lo);
          q1 = load_as_float(q + partner);
        }
        if constexpr (ROT) {
          if (u < half) {
            const float* turn = p.table + (t * half + u) * 2;
            turn_pair(k0, k1, turn[0], turn[1]);
            if constexpr (!SUMMARY) turn_pair(q0, q1, turn[0], turn[1]);
          }
        }
        Ks[row][lo] = k0 * live * p.k_scale;
        if (hi < Dk) Ks[row][hi] = k1 * live * p.k_scale;
        if constexpr (!SUMMARY) {
          Qs[row][lo] = q0 * live * p.q_scale;
          if (hi < Dk) Qs[row][hi] = q1 * live * p.q_scale;
        }
      }
    }
    // the chunk's decays: lane i of the first wave takes token i, a token that is not there adds nothing
    if (wave == 0) {
      const bool live = t0 + lane < end && lane < C;
      const float b = live ? (p.dt ? hr_softplus(dt_raw + p.dt_bias[h]) : 1.f) : 0.f;
      double sum = (double)b * rate;
#pragma unroll
      for (int step = 1; step < C; step *= 2) {
        const double other = __shfl_up(sum, step, 64);
        if (lane >= step) sum += other;
      }
      const double whole = __shfl(sum, C - 1, 64);
      if (lane < C) {
        sums[lane] = sum;
        scale_in[lane] = b;
        grow[lane] = exp2f((float)sum);
        weigh[lane] = exp2f((float)(whole - sum)) * b;
      }
    }
  };

  double total = 0.0;
  fetch(begin);
  for (int t0 = begin; t0 < end; t0 += C) {
    __syncthreads();               // the chunk before is consumed
    stage(t0);
    float v[8];
#pragma unroll
    for (int i = 0; i < 8; ++i)
      v[i] = (live_column && t0 + (i / 4) * 16 + lq * 4 + i % 4 < end) ? load_as_float(&v_raw[i]) : 0.f;
    __syncthreads();
    fetch(t0 + C);                 // in flight during this chunk's products (past the end the last token's again)

    if constexpr (!SUMMARY) {
      if (wave < 3) {              // scores of the tiles (0, 0), (1, 0) and (1, 1)
        const int it = wave > 0, jt = wave == 2;
        floatx4 score = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int t = 0; t < NT; ++t) {
          const floatx4 a = *(const floatx4*)&Qs[it * 16 + lr][t * 16 + lq * 4];
          const floatx4 b = *(const floatx4*)&Ks[jt * 16 + lr][t * 16 + lq * 4];
#pragma unroll
          for (int m = 0; m < 4; ++m) score = __builtin_amdgcn_mfma_f32_16x16x4f32(a[m], b[m], score, 0, 0, 0);
        }
        const int j = jt * 16 + lr;
        const double lj = sums[j];
        const float bj = scale_in[j];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int i = it * 16 + lq * 4 + r;
          Ps[i][j] = i >= j ? score[r] * exp2f((float)(sums[i] - lj)) * bj : 0.f;
        }
      }
      floatx4 o[2];
#pragma unroll
      for (int it = 0; it < 2; ++it) {
        o[it] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int t = 0; t < NT; ++t) {
          const floatx4 a = *(const floatx4*)&Qs[it * 16 + lr][t * 16 + lq * 4];
#pragma unroll
          for (int m = 0; m < 4; ++m) o[it] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[m], S[t][m], o[it], 0, 0, 0);
        }
        o[it] *= *(const floatx4*)&grow[it * 16 + lq * 4];
      }
      __syncthreads();             // the scores are there
#pragma unroll
      for (int it = 0; it < 2; ++it) {
#pragma unroll
        for (int jt = 0; jt <= it; ++jt) {
          const floatx4 a = *(const floatx4*)&Ps[it * 16 + lr][jt * 16 + lq * 4];
#pragma unroll
          for (int m = 0; m < 4; ++m) o[it] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[m], v[jt * 4 + m], o[it], 0, 0, 0);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int i = t0 + it * 16 + lq * 4 + r;
          if (live_column && i < end) p.out[((size_t)i * H + h) * Dv + column] = fmaf(skip, v[it * 4 + r], o[it][r]);
        }
      }
    }
    // the state moves past the chunk
    const float whole = grow[C - 1];
    if (SUMMARY) total += sums[C - 1];
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] *= weigh[(i / 4) * 16 + lq * 4 + i % 4];
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      S[t] *= whole;
#pragma unroll
      for (int i = 0; i < 8; ++i)
        S[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(Ks[(i / 4) * 16 + lq * 4 + i % 4][t * 16 + lr], v[i], S[t], 0, 0, 0);
    }
  }

  if (!SUMMARY && !last) return;
  float* to = SUMMARY ? p.seg_state + (((size_t)slot_index * H + h) * Dv + column_at) * Dk : home;
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = t * 16 + lq * 4 + r;
      if (live_column && d < Dk) to[d] = S[t][r];
    }
  if (SUMMARY && tid == 0 && column0 == 0) p.seg_sum[(size_t)slot_index * H + h] = total;
}

// From a sequence's state slot and its segments' summaries to the state ahead of every segment: a thread per
// (sequence, element of the state) chains them in order, each taking its summary's place.  (The first segment's
// is a copy of the slot: the slot itself is written by the block that walks the last segment.)
__global__ __launch_bounds__(HR_THREADS) void head_combine_kernel(HeadRecurrenceArgs p) {
  const int seq = blockIdx.y;
  const int begin = p.cu_q[seq], end = p.cu_q[seq + 1];
  const int slot = p.state_slots[seq];
  if (end <= begin || end > p.tokens || slot < 0 || slot >= p.slots) return;
  const int segments = (end - begin + p.seg_len - 1) / p.seg_len;
  const size_t each = (size_t)p.value_dim * p.key_dim, count = each * p.heads;
  const size_t e = (size_t)blockIdx.x * HR_THREADS + threadIdx.x;
  if (segments < 2 || e >= count) return;
  const int h = (int)(e / each);
  const size_t slot0 = (size_t)(begin / p.seg_len + seq);
  float s = p.state[(size_t)slot * count + e];
  for (int seg = 0; seg < segments; ++seg) {
    float* at = p.seg_state + (slot0 + seg) * count + e;
    const float own = seg + 1 < segments ? *at : 0.f;
    const float decay = seg + 1 < segments ? exp2f((float)p.seg_sum[(slot0 + seg) * p.heads + h]) : 0.f;
    *at = s;
    s = fmaf(decay, s, own);
  }
}

template <typename T, int NT, int VEC, bool ROT>
static void launch_prompt(const HeadRecurrenceArgs& p, int slots, hipStream_t stream) {
  const dim3 grid(p.heads * p.column_blocks, slots);
  if (p.seg_state) {
    head_recurrence_kernel<T, NT, VEC, ROT, true><<<grid, HR_THREADS, 0, stream>>>(p);
    const size_t count = (size_t)p.heads * p.value_dim * p.key_dim;
    head_combine_kernel<<<dim3((unsigned)((count + HR_THREADS - 1) / HR_THREADS), p.num_seqs), HR_THREADS, 0, stream>>>(p);
  }
  head_recurrence_kernel<T, NT, VEC, ROT, false><<<grid, HR_THREADS, 0, stream>>>(p);
}

template <typename T, bool ROT>
static void launch_sizes(const HeadRecurrenceArgs& p, bool wide, int slots, hipStream_t stream) {
  const int tiles = (p.key_dim + 15) / 16;
  if (!wide) {
    if (tiles <= 4) launch_prompt<T, 4, 1, ROT>(p, slots, stream);
    else launch_prompt<T, 16, 1, ROT>(p, slots, stream);
  } else if (tiles <= 2) launch_prompt<T, 2, 4, ROT>(p, slots, stream);
  else if (tiles <= 3) launch_prompt<T, 3, 4, ROT>(p, slots, stream);
  else if (tiles <= 4) launch_prompt<T, 4, 4, ROT>(p, slots, stream);
  else if (tiles <= 6) launch_prompt<T, 6, 4, ROT>(p, slots, stream);
  else if (tiles <= 8) launch_prompt<T, 8, 4, ROT>(p, slots, stream);
  else if (tiles <= 12) launch_prompt<T, 12, 4, ROT>(p, slots, stream);
  else launch_prompt<T, 16, 4, ROT>(p, slots, stream);
}

static bool aligned_rows(const void* p, size_t stride, size_t element) {
  return (uintptr_t)p % (4 * element) == 0 && stride % 4 == 0;
}

static int check_common(const HeadRecurrenceArgs& p, int dtype) {
  if (dtype != FE_F32 && dtype != FE_BF16) return FE_BAD_ARGUMENT;
  if (!p.q || !p.k || !p.v || !p.rate || !p.state || !p.cu_q || !p.state_slots) return FE_BAD_ARGUMENT;
  if (p.heads < 1 || p.share < 1 || p.heads % p.share || p.key_dim < 1 || p.key_dim > 256 || p.value_dim < 1 || p.slots < 1)
    return FE_BAD_ARGUMENT;
  const size_t shared = (size_t)(p.heads / p.share) * p.key_dim;
  if (p.q_stride < shared || p.k_stride < shared || p.v_stride < (size_t)p.heads * p.value_dim) return FE_BAD_ARGUMENT;
  if (p.rotary_dim < 0 || p.rotary_dim % 2 || p.rotary_dim > p.key_dim || (p.rotary_dim && !p.table)) return FE_BAD_ARGUMENT;
  if (p.dt && (!p.dt_bias || p.dt_stride < (size_t)p.heads)) return FE_BAD_ARGUMENT;
  return FE_OK;
}

// dtype: of q, k, v and dt (rows of any stride).  rate float32 [heads]: the logarithm of a head's decay, or with
// dt [tokens][heads] the (negative) factor on its step size.  out float32 [tokens][heads][value_dim], dense.
// seg_len: tokens a segment, a multiple of 32; with seg_state (float32 [slots of the launch][heads][value_dim]
// [key_dim]) and seg_sum (float64 [slots of the launch][heads]) a sequence longer than a segment is walked in segments
// side by side, slots of the launch >= tokens / seg_len + num_seqs; without them seg_len must be beyond the step.
extern "C" int fe_head_recurrence(const void* q, const void* k, const void* v, const void* dt, int dtype, long long q_stride,
                                  long long k_stride, long long v_stride, long long dt_stride, const float* table,
                                  int rotary_dim, const float* rate, const float* dt_bias, const float* skip, float q_scale,
                                  float k_scale, float* state, int slots, float* out, const int* cu_q,
                                  const int* state_slots, int num_seqs, int heads, int share, int key_dim, int value_dim,
                                  int tokens, int seg_len, float* seg_state, double* seg_sum, int seg_slots,
                                  hipStream_t stream) {
  if (tokens <= 0 || num_seqs <= 0) return FE_OK;
  HeadRecurrenceArgs p;
  p.q = q; p.k = k; p.v = v; p.dt = dt;
  p.q_stride = (size_t)q_stride; p.k_stride = (size_t)k_stride; p.v_stride = (size_t)v_stride; p.dt_stride = (size_t)dt_stride;
  p.table = table; p.rate = rate; p.dt_bias = dt_bias; p.skip = skip;
  p.state = state; p.out = out; p.seg_state = seg_state; p.seg_sum = seg_sum;
  p.cu_q = cu_q; p.state_slots = state_slots;
  p.q_scale = q_scale; p.k_scale = k_scale;
  p.rotary_dim = rotary_dim; p.heads = heads; p.share = share; p.key_dim = key_dim; p.value_dim = value_dim;
  p.tokens = tokens; p.num_seqs = num_seqs; p.slots = slots; p.seg_len = seg_len;
  p.column_blocks = (value_dim + HR_COLS - 1) / HR_COLS;
  const int status = check_common(p, dtype);
  if (status != FE_OK) return status;
  if (!out || seg_len < HR_CHUNK || seg_len % HR_CHUNK || (seg_state != nullptr) != (seg_sum != nullptr)) return FE_BAD_ARGUMENT;
  if (!seg_state && seg_len < tokens) return FE_BAD_ARGUMENT;
  const long long launch_slots = (long long)tokens / seg_len + num_seqs;
  if (launch_slots > 65535 || num_seqs > 65535 || (seg_state && seg_slots < launch_slots)) return FE_BAD_ARGUMENT;
  const size_t element = dtype == FE_F32 ? 4 : 2;
  const bool wide = key_dim % 8 == 0 && rotary_dim % 8 == 0 && aligned_rows(q, p.q_stride, element) &&
                    aligned_rows(k, p.k_stride, element) && (!rotary_dim || (uintptr_t)table % 16 == 0);
  if (dtype == FE_F32) {
    if (rotary_dim) launch_sizes<float, true>(p, wide, (int)launch_slots, stream);
    else launch_sizes<float, false>(p, wide, (int)launch_slots, stream);
  } else {
    if (rotary_dim) launch_sizes<bf16_t, true>(p, wide, (int)launch_slots, stream);
    else launch_sizes<bf16_t, false>(p, wide, (int)launch_slots, stream);
  }
  return fe_check_launch();
}

// ---------------------------------------------------------------- steps of single tokens
__device__ __forceinline__ float sum_16(float v) {
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0xB1, 0xF, 0xF, true));    // lane ^ 1
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x4E, 0xF, 0xF, true));    // lane ^ 2
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x141, 0xF, 0xF, true));   // 7 - lane within 8
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x140, 0xF, 0xF, true));   // 15 - lane within 16
  return v;
}

#define HS_THREADS 512
#define HS_COLUMNS (HS_THREADS / 16)      // columns the block takes at a time
#define HS_AHEAD 4                        // ... and how many such rounds have their loads in flight together
#define HS_MAX_NORMED 1024                // widest head whose read-out is kept for its norm

// Lane s of a column holds key dims 4 s + 64 m .. + 3 for m < NM (VEC 4; loads of 16 bytes) or the same dims one by
// one.  GATED: the block takes all columns of the head and ends with the norm and the gate (out in T), else
// blockIdx.z takes a run of columns and out is float32.
template <typename T, int NM, bool VEC, bool GATED>
__global__ __launch_bounds__(HS_THREADS) void head_recurrence_step_kernel(HeadRecurrenceArgs p, const T* __restrict__ gate,
                                                                          size_t gate_stride, T* __restrict__ normed,
                                                                          size_t normed_stride, float eps, int columns_each) {
  __shared__ __attribute__((aligned(16))) float qs[256], ks[256];
  __shared__ float ys[GATED ? HS_MAX_NORMED : 1];
  __shared__ float scratch[16];
  const int h = blockIdx.x, seq = blockIdx.y, tid = threadIdx.x;
  const int t = p.cu_q[seq];
  const int slot = p.state_slots[seq];
  if (p.cu_q[seq + 1] != t + 1 || t >= p.tokens || slot < 0 || slot >= p.slots) return;
  const int Dk = p.key_dim, Dv = p.value_dim, H = p.heads;
  const int first = blockIdx.z * columns_each, stop = min(Dv, first + columns_each);
  const int lane16 = tid % 16, column_of = tid / 16;
  float* home = p.state + ((size_t)slot * H + h) * Dv * Dk;

  floatx4 S[HS_AHEAD][NM];
  float v[HS_AHEAD];
  auto load = [&](int c0) {
#pragma unroll
    for (int a = 0; a < HS_AHEAD; ++a) {
      const int column = min(c0 + a * HS_COLUMNS + column_of, Dv - 1);
      const float* row = home + (size_t)column * Dk;
#pragma unroll
      for (int m = 0; m < NM; ++m) {
        const int d = lane16 * 4 + m * 64;
        if constexpr (VEC) {
          S[a][m] = *(const floatx4*)(row + min(d, Dk - 4));
        } else {
#pragma unroll
          for (int i = 0; i < 4; ++i) S[a][m][i] = row[min(d + i, Dk - 1)];
        }
      }
      v[a] = load_as_float((const T*)p.v + (size_t)t * p.v_stride + (size_t)h * Dv + column);
    }
  };
  load(first);

  const size_t head_at = (size_t)(h / p.share) * Dk;
  const int half = p.rotary_dim / 2;
  if (tid < 256) {
    const int d = tid;
    float q = 0.f, k = 0.f;
    if (d < Dk) {
      const T* qrow = (const T*)p.q + (size_t)t * p.q_stride + head_at;
      const T* krow = (const T*)p.k + (size_t)t * p.k_stride + head_at;
      q = load_as_float(qrow + d);
      k = load_as_float(krow + d);
      if (d < 2 * half) {
        const int pair = d < half ? d : d - half;
        const float cs = p.table[((size_t)t * half + pair) * 2];
        const float sn = d < half ? -p.table[((size_t)t * half + pair) * 2 + 1] : p.table[((size_t)t * half + pair) * 2 + 1];
        const int other = d < half ? d + half : d - half;
        q = q * cs + load_as_float(qrow + other) * sn;
        k = k * cs + load_as_float(krow + other) * sn;
      }
    }
    qs[d] = q * p.q_scale;
    ks[d] = k * p.k_scale;
  }
  const float b = p.dt ? hr_softplus(load_as_float((const T*)p.dt + (size_t)t * p.dt_stride + h) + p.dt_bias[h]) : 1.f;
  const float decay = exp2f((float)((double)b * (double)p.rate[h] * HR_LOG2E));
  const float skip = p.skip ? p.skip[h] : 0.f;
  __syncthreads();

  floatx4 q[NM], k[NM];
#pragma unroll
  for (int m = 0; m < NM; ++m) {
    q[m] = *(const floatx4*)&qs[lane16 * 4 + m * 64];
    k[m] = *(const floatx4*)&ks[lane16 * 4 + m * 64];
  }
  float squares = 0.f;
  for (int c0 = first; c0 < stop; c0 += HS_COLUMNS * HS_AHEAD) {
    if (c0 > first) load(c0);
#pragma unroll
    for (int a = 0; a < HS_AHEAD; ++a) {
      const int column = c0 + a * HS_COLUMNS + column_of;
      const float bv = b * v[a];
      float y = 0.f;
#pragma unroll
      for (int m = 0; m < NM; ++m)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          S[a][m][i] = fmaf(S[a][m][i], decay, k[m][i] * bv);
          y = fmaf(S[a][m][i], q[m][i], y);        // dims beyond the real ones meet q = 0
        }
      if (column < stop) {
        float* row = home + (size_t)column * Dk;
#pragma unroll
        for (int m = 0; m < NM; ++m) {
          const int d = lane16 * 4 + m * 64;
          if constexpr (VEC) {
            if (d < Dk) *(floatx4*)(row + d) = S[a][m];
          } else {
#pragma unroll
            for (int i = 0; i < 4; ++i)
              if (d + i < Dk) row[d + i] = S[a][m][i];
          }
        }
      }
      y = fmaf(skip, v[a], sum_16(y));
      if (column < stop && lane16 == 0) {
        if constexpr (GATED) {
          ys[column] = y;
          squares = fmaf(y, y, squares);
        } else {
          p.out[((size_t)t * H + h) * Dv + column] = y;
        }
      }
    }
  }
  if constexpr (GATED) {
    const float inv = rsqrtf(block_sum<true>(squares, scratch) / (float)Dv + eps);
    for (int c = tid; c < Dv; c += HS_THREADS) {
      const float g = load_as_float(gate + (size_t)t * gate_stride + (size_t)h * Dv + c);
      store_from_float(normed + (size_t)t * normed_stride + (size_t)h * Dv + c, ys[c] * inv * hr_silu(g));
    }
  }
}

template <typename T, int NM>
static void launch_step(const HeadRecurrenceArgs& p, const void* gate, size_t gate_stride, void* normed, size_t normed_stride,
                        float eps, hipStream_t stream) {
  const bool vec = p.key_dim % 4 == 0;
  const int columns_each = gate ? p.value_dim : HS_COLUMNS * HS_AHEAD;
  const dim3 grid(p.heads, p.num_seqs, (p.value_dim + columns_each - 1) / columns_each);
#define LAUNCH(VEC, GATED)                                                                                            \
  head_recurrence_step_kernel<T, NM, VEC, GATED><<<grid, HS_THREADS, 0, stream>>>(p, (const T*)gate, gate_stride, (T*)normed, \
                                                                                  normed_stride, eps, columns_each)
  if (gate) {
    if (vec) LAUNCH(true, true); else LAUNCH(false, true);
  } else {
    if (vec) LAUNCH(true, false); else LAUNCH(false, false);
  }
#undef LAUNCH
}

// Every sequence brings one token (others are left alone).  Without a gate: out as above.  With a gate ([tokens]
// rows of heads * value_dim, value_dim <= 1024): normed[t][h] = o / sqrt(mean(o^2) + eps) * silu(gate), in dtype.
extern "C" int fe_head_recurrence_step(const void* q, const void* k, const void* v, const void* dt, int dtype,
                                       long long q_stride, long long k_stride, long long v_stride, long long dt_stride,
                                       const float* table, int rotary_dim, const float* rate, const float* dt_bias,
                                       const float* skip, float q_scale, float k_scale, float* state, int slots, float* out,
                                       const void* gate, long long gate_stride, void* normed, long long normed_stride,
                                       float eps, const int* cu_q, const int* state_slots, int num_seqs, int heads, int share,
                                       int key_dim, int value_dim, int tokens, hipStream_t stream) {
  if (tokens <= 0 || num_seqs <= 0) return FE_OK;
  HeadRecurrenceArgs p = {};
  p.q = q; p.k = k; p.v = v; p.dt = dt;
  p.q_stride = (size_t)q_stride; p.k_stride = (size_t)k_stride; p.v_stride = (size_t)v_stride; p.dt_stride = (size_t)dt_stride;
  p.table = table; p.rate = rate; p.dt_bias = dt_bias; p.skip = skip;
  p.state = state; p.out = out; p.cu_q = cu_q; p.state_slots = state_slots;
  p.q_scale = q_scale; p.k_scale = k_scale;
  p.rotary_dim = rotary_dim; p.heads = heads; p.share = share; p.key_dim = key_dim; p.value_dim = value_dim;
  p.tokens = tokens; p.num_seqs = num_seqs; p.slots = slots;
  const int status = check_common(p, dtype);
  if (status != FE_OK) return status;
  if (num_seqs > 65535 || (!gate && !out)) return FE_BAD_ARGUMENT;
  if (gate && (!normed || value_dim > HS_MAX_NORMED || !(eps > 0.f) || gate_stride < (long long)heads * value_dim ||
               normed_stride < (long long)heads * value_dim))
    return FE_BAD_ARGUMENT;
#define STEP(T)                                                                                                         \
  do {                                                                                                                  \
    if (key_dim <= 64) launch_step<T, 1>(p, gate, (size_t)gate_stride, normed, (size_t)normed_stride, eps, stream);     \
    else if (key_dim <= 128) launch_step<T, 2>(p, gate, (size_t)gate_stride, normed, (size_t)normed_stride, eps, stream); \
    else if (key_dim <= 192) launch_step<T, 3>(p, gate, (size_t)gate_stride, normed, (size_t)normed_stride, eps, stream); \
    else launch_step<T, 4>(p, gate, (size_t)gate_stride, normed, (size_t)normed_stride, eps, stream);                   \
  } while (0)
  if (dtype == FE_F32) STEP(float);
  else STEP(bf16_t);
#undef STEP
  return fe_check_launch();
}

// ---------------------------------------------------------------- tables of cosines and sines
// table[t][i] = (cos, sin)(position_t * inv_freq[i]): one a step, for every mixer that turns by the same frequencies.
__global__ void rotary_table_kernel(const int* __restrict__ positions, const float* __restrict__ inv_freq,
                                    float2* __restrict__ table, int half, long long count) {
  const long long e = (long long)blockIdx.x * blockDim.x + threadIdx.x;
  if (e >= count) return;
  float sn, cs;
  sincosf((float)positions[e / half] * inv_freq[e % half], &sn, &cs);
  table[e] = make_float2(cs, sn);
}

extern "C" int fe_rotary_table(const int* positions, const float* inv_freq, float* table, int tokens, int half,
                               hipStream_t stream) {
  if (tokens <= 0) return FE_OK;
  if (half < 1 || !positions || !inv_freq || !table) return FE_BAD_ARGUMENT;
  const long long count = (long long)tokens * half;
  rotary_table_kernel<<<(unsigned)((count + 255) / 256), 256, 0, stream>>>(positions, inv_freq, (float2*)table, half, count);
  return fe_check_launch();
}
