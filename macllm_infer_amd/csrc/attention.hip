// Rotary position encoding fused with the write of K and V into cache pages, and
// attention over the paged cache.
//
// Cache layout of one paged group: [page, layer, 2 (K,V), kv_head, page_size*head_dim].
// Inside a page, K of one kv head is [token, dim] and V is transposed, [dim, token]: the
// value product contracts over tokens, and a matrix-core operand wants its contraction index
// contiguous.  Entry points get the base pointers of one layer's K and V inside page 0 and
// the stride between pages:
//   K(page, kvh, off, i) = k_base + page*page_stride + (kvh*page_size + off)*dh + i
//   V(page, kvh, off, i) = v_base + page*page_stride + (kvh*dv + i)*page_size + off
// with dv the width of a value head, which the general kernels take apart from dh, the width of a key head.
// (The reference pages its cache the same way, K and V both token-major:
// crates/macllm-kv/src/cache.rs:558-566, crates/macllm-kernels/src/metal/paged_decode.metal:109-113.)
#include "common.h"
#include <type_traits>

// ---------------------------------------------------------------- rope + cache write
// For token t at absolute position p:
//   q[t, h, :] is rotated in place; k[t, h, :] is rotated and stored; v[t, h, :] is stored.
//   Rotation (half-split, first rotary_dim dims): angle = (float)p * inv_freq[j];
//   out[j] = x[j] cos - x[j+half] sin;  out[j+half] = x[j+half] cos + x[j] sin.
//   (reference: src/decoder.rs:186-195, 226-229; K is cached after rotation, :953-962)
// slot_mapping[t] = page*page_size + offset of the token's cache cell; null = nothing is stored.
template <typename T>
__global__ void rope_kv_store_kernel(T* __restrict__ qkv, long ld, int Hq, int Hkv, int dh, int dv,
                                     const int* __restrict__ positions, const float* __restrict__ inv_freq,
                                     int rotary_dim, const int* __restrict__ slot_mapping,
                                     T* __restrict__ k_base, T* __restrict__ v_base, long page_stride,
                                     int page_size) {
  const long token = blockIdx.x;
  T* row = qkv + token * ld;
  const float position = (float)positions[token];
  const int half = rotary_dim / 2;
  long cell = -1;
  long page = 0;
  int offset = 0;
  if (slot_mapping) {
    cell = slot_mapping[token];
    page = cell / page_size;
    offset = (int)(cell - page * page_size);
  }
  // q heads then k heads: (head, pair) items
  const int rotary_heads = Hq + Hkv;
  const int pairs = rotary_heads * (dh / 2);   // items cover dh/2 "columns": rotated pairs and pass-through pairs
  for (int item = threadIdx.x; item < pairs; item += blockDim.x) {
    const int head = item / (dh / 2);
    const int j = item - head * (dh / 2);
    T* x = row + (long)head * dh;
    // column j pairs with j+half when j < half; columns >= rotary_dim pass through.
    // Enumerate so that every element of the head is visited exactly once:
    //   j in [0, half): rotated pair (j, j+half)
    //   j in [half, dh/2): pass-through elements (rotary_dim + 2*(j-half)) and the next one
    float a, b;
    int ia, ib;
    if (j < half) {
      ia = j;
      ib = j + half;
      const float x0 = to_float(x[ia]);
      const float x1 = to_float(x[ib]);
      float s = 0.f, c = 1.f;
      if (inv_freq) {
        const float angle = position * inv_freq[j];
        s = sinf(angle);
        c = cosf(angle);
      }
      a = x0 * c - x1 * s;
      b = x1 * c + x0 * s;
    } else {
      ia = rotary_dim + 2 * (j - half);
      ib = ia + 1;
      a = to_float(x[ia]);
      b = to_float(x[ib]);
    }
    if (head < Hq) {
      x[ia] = from_float<T>(a);
      x[ib] = from_float<T>(b);
    } else if (cell >= 0) {
      const int kvh = head - Hq;
      T* dst = k_base + page * page_stride + ((long)kvh * page_size + offset) * dh;
      dst[ia] = from_float<T>(a);
      dst[ib] = from_float<T>(b);
    }
  }
  if (cell >= 0) {
    const T* v = row + (long)(Hq + Hkv) * dh;
    for (int item = threadIdx.x; item < Hkv * dv; item += blockDim.x) {
      const int kvh = item / dv;
      const int i = item - kvh * dv;
      v_base[page * page_stride + ((long)kvh * dv + i) * page_size + offset] = v[item];
    }
  }
}

// dv: the width of a value head (the v heads follow the k heads in a row of qkv).
extern "C" int mi_rope_kv_store(void* qkv, int dtype, long ld, int T, int Hq, int Hkv, int dh, int dv,
                                const int* positions, const float* inv_freq, int rotary_dim,
                                const int* slot_mapping, void* k_base, void* v_base, long page_stride,
                                int page_size, hipStream_t stream) {
  if (T <= 0 || Hq <= 0 || Hkv <= 0 || dh <= 0 || (dh & 1) || dv <= 0) return ERR_BAD_ARGUMENT;
  if (rotary_dim < 0 || rotary_dim > dh || (rotary_dim & 1)) return ERR_BAD_ARGUMENT;
  if (ld < (long)(Hq + Hkv) * dh + (long)Hkv * dv) return ERR_BAD_ARGUMENT;
  if (slot_mapping && (!k_base || !v_base || page_size <= 0)) return ERR_BAD_ARGUMENT;
  if (!inv_freq) rotary_dim = 0;
  if (dtype == DT_F32)
    rope_kv_store_kernel<float><<<T, 256, 0, stream>>>((float*)qkv, ld, Hq, Hkv, dh, dv, positions, inv_freq,
                                                        rotary_dim, slot_mapping, (float*)k_base,
                                                        (float*)v_base, page_stride, page_size);
  else if (dtype == DT_BF16)
    rope_kv_store_kernel<bf16_t><<<T, 256, 0, stream>>>((bf16_t*)qkv, ld, Hq, Hkv, dh, dv, positions, inv_freq,
                                                         rotary_dim, slot_mapping, (bf16_t*)k_base,
                                                         (bf16_t*)v_base, page_stride, page_size);
  else
    return ERR_BAD_ARGUMENT;
  RETURN_IF_LAUNCH_FAILED();
  return 0;
}

// ---------------------------------------------------------------- a token's row made ready for attention
// One workgroup a token; the row [q heads | k heads | v heads] is laid in LDS as float32 and everything below is
// float32 arithmetic on that copy:
//   * q_norm / k_norm (optional): the whole q projection (Hq * dh numbers), and the whole k projection, is divided by
//     its root mean square (eps inside the root) and multiplied by a weight of that length, before rotation;
//   * head_norm (1: before the rotation, 2: after it): every q head and every k head is divided by its own root mean
//     square over dh (head_eps inside the root) and multiplied by q_head_weight / k_head_weight (float32 [dh], one
//     weight for all heads; null: the bare division);
//   * q and k are turned by the token's position over the first rotary_dim dims, angle = (float)position *
//     inv_freq[j], pairs (j, j + rotary_dim / 2) or, interleaved, (2j, 2j + 1); cosines and sines times turn_scale;
//     q is written back in place, k goes to the token's cache cell;
//   * with temp_every > 0 the queries are multiplied by 1 + temp_coef * ln(floor((position + 1) / temp_every) + 1);
//   * the values are the v heads of the row or, with values_from_keys, the k heads as they were projected (before
//     norm and rotation; dv = dh); with value_inv_freq they are turned by the position over all dv dims (half-split
//     pairs, angle = (float)position * value_inv_freq[m]); they go to the token's transposed cache cell.
// A row of queries alone (Hkv = 0, no slot_mapping) is one whose keys and values another layer has cached.
template <typename T>
__global__ void __launch_bounds__(256)
attention_prepare_kernel(T* __restrict__ qkv, long ld, int Hq, int Hkv, int dh, int dv, int values_from_keys,
                         const int* __restrict__ positions, const float* __restrict__ inv_freq, int rotary_dim,
                         int interleaved, float turn_scale,
                         const float* __restrict__ q_norm, const float* __restrict__ k_norm, float norm_eps,
                         int head_norm, const float* __restrict__ q_head_weight, const float* __restrict__ k_head_weight,
                         float head_eps, float temp_coef, int temp_every,
                         const float* __restrict__ value_inv_freq, const int* __restrict__ slot_mapping,
                         T* __restrict__ k_base, T* __restrict__ v_base, long page_stride, int page_size) {
  extern __shared__ float prepared_row[];
  __shared__ float scratch[16];
  const long token = blockIdx.x;
  T* row = qkv + token * ld;
  const float position = (float)positions[token];
  const int q_cols = Hq * dh, k_cols = Hkv * dh;
  const int v_cols = Hkv * dv;
  float* q_lds = prepared_row;
  float* k_lds = q_lds + q_cols;
  float* v_lds = k_lds + k_cols;
  // the token's turns, (cosine, sine) a pair of dims, once for all heads: keys' pairs, then the values'
  const int half = rotary_dim / 2;
  const int value_half = dv / 2;
  float* turns = v_lds + v_cols;
  float* value_turns = turns + 2 * half;
  if (inv_freq)
    for (int j = threadIdx.x; j < half; j += blockDim.x) {
      float sine, cosine;
      sincosf(position * inv_freq[j], &sine, &cosine);
      turns[2 * j] = cosine * turn_scale;
      turns[2 * j + 1] = sine * turn_scale;
    }
  if (value_inv_freq)
    for (int m = threadIdx.x; m < value_half; m += blockDim.x) {
      float sine, cosine;
      sincosf(position * value_inv_freq[m], &sine, &cosine);
      value_turns[2 * m] = cosine;
      value_turns[2 * m + 1] = sine;
    }
  float q_squares = 0.f, k_squares = 0.f;
  for (int i = threadIdx.x; i < q_cols + k_cols; i += blockDim.x) {
    const float x = to_float(row[i]);
    prepared_row[i] = x;
    if (i < q_cols) q_squares = fmaf(x, x, q_squares);
    else k_squares = fmaf(x, x, k_squares);
  }
  for (int i = threadIdx.x; i < v_cols; i += blockDim.x)
    v_lds[i] = to_float(values_from_keys ? row[q_cols + i] : row[q_cols + k_cols + i]);
  if (q_norm) {
    const float q_rms = sqrtf(block_sum(q_squares, scratch) / (float)q_cols + norm_eps);
    const float k_rms = sqrtf(block_sum(k_squares, scratch) / (float)k_cols + norm_eps);
    for (int i = threadIdx.x; i < q_cols; i += blockDim.x) q_lds[i] = q_lds[i] / q_rms * q_norm[i];
    for (int i = threadIdx.x; i < k_cols; i += blockDim.x) k_lds[i] = k_lds[i] / k_rms * k_norm[i];
  }
  __syncthreads();
  // a head's root mean square: one wave a head, the lanes' shares added in an order that dh alone fixes
  auto norm_heads = [&]() {
    const int lane = threadIdx.x & (WAVE - 1);
    const int waves = blockDim.x / WAVE;
    for (int head = threadIdx.x / WAVE; head < Hq + Hkv; head += waves) {
      float* x = prepared_row + (long)head * dh;
      const float* weight = head < Hq ? q_head_weight : k_head_weight;
      float squares = 0.f;
      for (int j = lane; j < dh; j += WAVE) squares = fmaf(x[j], x[j], squares);
      const float rms = sqrtf(wave_sum(squares) / (float)dh + head_eps);
      for (int j = lane; j < dh; j += WAVE) x[j] = weight ? x[j] / rms * weight[j] : x[j] / rms;
    }
    __syncthreads();
  };
  if (head_norm == 1) norm_heads();
  // q heads then k heads: a thread a pair of dims, turned in place in LDS
  if (inv_freq && half > 0) {
    for (int item = threadIdx.x; item < (Hq + Hkv) * half; item += blockDim.x) {
      const int head = item / half;
      const int pair = item - head * half;
      float* x = prepared_row + (long)head * dh;
      const int ia = interleaved ? 2 * pair : pair;
      const int ib = interleaved ? 2 * pair + 1 : pair + half;
      const float cosine = turns[2 * pair], sine = turns[2 * pair + 1];
      const float u = x[ia], v = x[ib];
      x[ia] = u * cosine - v * sine;
      x[ib] = v * cosine + u * sine;
    }
    __syncthreads();
  }
  if (head_norm == 2) norm_heads();
  const float temperature = temp_every > 0 ? 1.0f + temp_coef * logf((float)((positions[token] + 1) / temp_every + 1)) : 1.0f;
  long cell = -1, page = 0;
  int offset = 0;
  if (slot_mapping) {
    cell = slot_mapping[token];
    page = cell / page_size;
    offset = (int)(cell - page * page_size);
  }
  for (int item = threadIdx.x; item < q_cols + k_cols; item += blockDim.x) {
    const int head = item / dh;
    const int j = item - head * dh;
    const float value = prepared_row[item];
    if (head < Hq) row[item] = from_float<T>(value * temperature);
    else if (cell >= 0)
      k_base[page * page_stride + ((long)(head - Hq) * page_size + offset) * dh + j] = from_float<T>(value);
  }
  if (cell >= 0) {
    for (int item = threadIdx.x; item < v_cols; item += blockDim.x) {
      const int kvh = item / dv;
      const int i = item - kvh * dv;
      float value = v_lds[item];
      if (value_inv_freq) {
        const bool low = i < value_half;
        const int pair = low ? i : i - value_half;
        const float cosine = value_turns[2 * pair], sine = value_turns[2 * pair + 1];
        const float partner = v_lds[kvh * dv + (low ? i + value_half : i - value_half)];
        value = low ? value * cosine - partner * sine : value * cosine + partner * sine;
      }
      v_base[page * page_stride + ((long)kvh * dv + i) * page_size + offset] = from_float<T>(value);
    }
  }
}

// The same where no norm spans a whole projection: everything is then head by head, and a wave makes one head ready by
// itself (grid: tokens x fours of [q heads | k heads | v heads]), its elements in registers, a lane the elements lane,
// lane + 64, ...; a pair's partner comes through the wave's own row of LDS.  The sums are the ones of the kernel above.
#define PREPARE_WAVES 4
#define PREPARE_PER_LANE 4       // heads of up to 256 dims
#define PREPARE_HEADS_TOKENS 512
template <typename T>
__global__ void __launch_bounds__(PREPARE_WAVES * WAVE)
attention_prepare_heads_kernel(T* __restrict__ qkv, long ld, int Hq, int Hkv, int dh, int dv, int values_from_keys,
                               const int* __restrict__ positions, const float* __restrict__ inv_freq, int rotary_dim,
                               int interleaved, float turn_scale, int head_norm, const float* __restrict__ q_head_weight,
                               const float* __restrict__ k_head_weight, float head_eps, float temp_coef, int temp_every,
                               const float* __restrict__ value_inv_freq, const int* __restrict__ slot_mapping,
                               T* __restrict__ k_base, T* __restrict__ v_base, long page_stride, int page_size) {
  __shared__ float rows[PREPARE_WAVES][WAVE * PREPARE_PER_LANE];
  const long token = blockIdx.x;
  const int lane = threadIdx.x & (WAVE - 1);
  const int wave = threadIdx.x / WAVE;
  const int index = blockIdx.y * PREPARE_WAVES + wave;              // q heads, k heads, v heads
  if (index >= Hq + 2 * Hkv) return;                                 // (no barrier of the workgroup below)
  const bool is_q = index < Hq;
  const bool is_v = index >= Hq + Hkv;
  const int kvh = is_v ? index - Hq - Hkv : index - Hq;
  const int width = is_v ? dv : dh;
  const int place = positions[token];
  const float position = (float)place;
  const int cell = slot_mapping ? slot_mapping[token] : -1;
  T* row = qkv + token * ld;
  T* from = row;
  if (is_q) from += (long)index * dh;
  else if (!is_v || values_from_keys) from += (long)(Hq + kvh) * dh;
  else from += (long)(Hq + Hkv) * dh + (long)kvh * dv;
  const float* weight = is_v ? nullptr : is_q ? q_head_weight : k_head_weight;
  const int turned = is_v ? (value_inv_freq ? dv : 0) : (inv_freq ? rotary_dim : 0);
  const float* frequencies = is_v ? value_inv_freq : inv_freq;
  const float magnitude = is_v ? 1.0f : turn_scale;
  const bool neighbours = !is_v && interleaved;
  const int norm = is_v ? 0 : head_norm;
  float x[PREPARE_PER_LANE], w[PREPARE_PER_LANE];
#pragma unroll
  for (int i = 0; i < PREPARE_PER_LANE; ++i) {
    const int j = lane + WAVE * i;
    x[i] = j < width ? to_float(from[j]) : 0.f;
    w[i] = (weight && j < width) ? weight[j] : 1.f;
  }
  auto norm_head = [&]() {
    float squares = 0.f;
#pragma unroll
    for (int i = 0; i < PREPARE_PER_LANE; ++i) squares = fmaf(x[i], x[i], squares);
    const float rms = sqrtf(wave_sum(squares) / (float)dh + head_eps);
#pragma unroll
    for (int i = 0; i < PREPARE_PER_LANE; ++i) x[i] = weight ? x[i] / rms * w[i] : x[i] / rms;
  };
  if (norm == 1) norm_head();
  if (turned > 0) {
    const int half = turned / 2;
    float* mine = rows[wave];
#pragma unroll
    for (int i = 0; i < PREPARE_PER_LANE; ++i) mine[lane + WAVE * i] = x[i];
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int i = 0; i < PREPARE_PER_LANE; ++i) {
      const int j = lane + WAVE * i;
      if (j < turned) {
        const int pair = neighbours ? j / 2 : (j < half ? j : j - half);
        const bool first = neighbours ? (j & 1) == 0 : j < half;
        const float partner = mine[neighbours ? (j ^ 1) : (first ? j + half : j - half)];
        float sine, cosine;
        sincosf(position * frequencies[pair], &sine, &cosine);
        sine *= magnitude;
        cosine *= magnitude;
        x[i] = first ? x[i] * cosine - partner * sine : x[i] * cosine + partner * sine;
      }
    }
  }
  if (norm == 2) norm_head();
  if (is_q) {
    const float temperature = temp_every > 0 ? 1.0f + temp_coef * logf((float)((place + 1) / temp_every + 1)) : 1.0f;
#pragma unroll
    for (int i = 0; i < PREPARE_PER_LANE; ++i) {
      const int j = lane + WAVE * i;
      if (j < width) from[j] = from_float<T>(x[i] * temperature);
    }
    return;
  }
  if (cell < 0) return;
  const int page = cell / page_size;
  const int offset = cell - page * page_size;
  T* to = is_v ? v_base + (long)page * page_stride + (long)kvh * dv * page_size + offset
               : k_base + (long)page * page_stride + ((long)kvh * page_size + offset) * dh;
  const int step = is_v ? page_size : 1;
#pragma unroll
  for (int i = 0; i < PREPARE_PER_LANE; ++i) {
    const int j = lane + WAVE * i;
    if (j < width) to[(long)j * step] = from_float<T>(x[i]);
  }
}

extern "C" int mi_attention_prepare(void* qkv, int dtype, long ld, int T, int Hq, int Hkv, int dh, int dv,
                                    int values_from_keys, const int* positions, const float* inv_freq, int rotary_dim,
                                    int interleaved, float turn_scale,
                                    const float* q_norm, const float* k_norm, float norm_eps,
                                    int head_norm, const float* q_head_weight, const float* k_head_weight, float head_eps,
                                    float temp_coef, int temp_every, const float* value_inv_freq, const int* slot_mapping, void* k_base, void* v_base,
                                    long page_stride, int page_size, hipStream_t stream) {
  if (!qkv || !positions || T <= 0 || Hq <= 0 || Hkv < 0 || dh <= 0 || dv <= 0 || temp_every < 0) return ERR_BAD_ARGUMENT;
  if (Hkv == 0 && (slot_mapping || q_norm || values_from_keys)) return ERR_BAD_ARGUMENT;      // queries alone
  if (rotary_dim < 0 || rotary_dim > dh || (rotary_dim & 1) || (rotary_dim > 0 && !inv_freq)) return ERR_BAD_ARGUMENT;
  if (values_from_keys && dv != dh) return ERR_BAD_ARGUMENT;
  if (value_inv_freq && (dv & 1)) return ERR_BAD_ARGUMENT;
  if ((q_norm == nullptr) != (k_norm == nullptr)) return ERR_BAD_ARGUMENT;
  if (head_norm < 0 || head_norm > 2 || (head_norm && q_norm) || (head_norm && !(head_eps > 0.f))) return ERR_BAD_ARGUMENT;
  if ((q_head_weight == nullptr) != (k_head_weight == nullptr) || (q_head_weight && !head_norm)) return ERR_BAD_ARGUMENT;
  if (ld < (long)(Hq + Hkv) * dh + (values_from_keys ? 0L : (long)Hkv * dv)) return ERR_BAD_ARGUMENT;
  if (slot_mapping && (!k_base || !v_base || page_size <= 0)) return ERR_BAD_ARGUMENT;
  if (!inv_freq) rotary_dim = 0;
  // few tokens wait for a chain of loads, which is shortest head by head; many tokens share a row's turns
  if (!q_norm && T <= PREPARE_HEADS_TOKENS && dh <= WAVE * PREPARE_PER_LANE && dv <= WAVE * PREPARE_PER_LANE) {
    const int items = slot_mapping ? Hq + 2 * Hkv : Hq;      // without cells the keys and values go nowhere
    const dim3 grid(T, (items + PREPARE_WAVES - 1) / PREPARE_WAVES);
#define PREPARE_HEADS(T_)                                                                                                   \
  attention_prepare_heads_kernel<T_><<<grid, PREPARE_WAVES * WAVE, 0, stream>>>(                                            \
      (T_*)qkv, ld, Hq, slot_mapping ? Hkv : 0, dh, dv, values_from_keys, positions, inv_freq, rotary_dim, interleaved,     \
      turn_scale, head_norm, q_head_weight, k_head_weight, head_eps, temp_coef, temp_every, value_inv_freq, slot_mapping,   \
      (T_*)k_base, (T_*)v_base, page_stride, page_size)
    if (dtype == DT_F32) PREPARE_HEADS(float);
    else if (dtype == DT_BF16) PREPARE_HEADS(bf16_t);
    else return ERR_BAD_ARGUMENT;
#undef PREPARE_HEADS
    RETURN_IF_LAUNCH_FAILED();
    return 0;
  }
  // the row, and (cosine, sine) of the keys' and the values' pairs
  const size_t lds = ((size_t)(Hq + Hkv) * dh + (size_t)Hkv * dv + (size_t)rotary_dim + (size_t)(dv / 2) * 2) * sizeof(float);
  if (lds > 64 * 1024) return ERR_UNSUPPORTED_SIZE;
  if (dtype == DT_F32)
    attention_prepare_kernel<float><<<T, 256, lds, stream>>>((float*)qkv, ld, Hq, Hkv, dh, dv, values_from_keys, positions,
                                                             inv_freq, rotary_dim, interleaved, turn_scale, q_norm, k_norm,
                                                             norm_eps, head_norm, q_head_weight, k_head_weight, head_eps,
                                                             temp_coef, temp_every, value_inv_freq, slot_mapping, (float*)k_base, (float*)v_base,
                                                             page_stride, page_size);
  else if (dtype == DT_BF16)
    attention_prepare_kernel<bf16_t><<<T, 256, lds, stream>>>((bf16_t*)qkv, ld, Hq, Hkv, dh, dv, values_from_keys,
                                                              positions, inv_freq, rotary_dim, interleaved, turn_scale,
                                                              q_norm, k_norm, norm_eps, head_norm, q_head_weight,
                                                              k_head_weight, head_eps, temp_coef, temp_every, value_inv_freq, slot_mapping,
                                                              (bf16_t*)k_base, (bf16_t*)v_base, page_stride, page_size);
  else
    return ERR_BAD_ARGUMENT;
  RETURN_IF_LAUNCH_FAILED();
  return 0;
}

// ---------------------------------------------------------------- paged attention, any size
// Works for any head_dim <= 256, any page size, any group size, float32 and bfloat16; the float32 path of
// the whole model uses it for prompts and for decoding alike.
//   s = q.k * scale;  visible keys: position <= query position, and
//   query - key < window when window > 0 (reference: src/decoder.rs:4515-4532), or of the query's own chunk of
//   -window positions when window < 0 (first_visible_key); with kept > 0 the keys at
//   positions below kept stay visible behind the window (the first tokens of a sequence, at their true positions);
//   softmax in float32 (reference: src/decoder.rs:4665-4667).
// `slopes` (optional, float32 per query head): a position encoding that is a bias on the scores,
//   s -= slopes[head] * (query position - key position)   (no counterpart in the reference).
// `log_bias` (optional, float32 [query heads][2] = (r1, r2)): a bias that grows with the logarithm of the distance,
//   s -= r1 * ln(1 + r2 * (query position - key position)).
// `sinks` (optional, float32 per query head, read by the merge kernel): exp(sink) is one more term of the softmax's
//   denominator; it has no key and no value.
// `head_scales` (optional, float32 per query head): s *= head_scales[head] behind the scale.
// `sigmoid` (with an optional `score_bias`, float32 per query head): a visible key weighs sigmoid(s + score_bias[head])
//   on its own and nothing is normalized: the kernels keep the maximum 0 for every group of keys, so every weight of
//   the merges below is exp(0) = 1 and the sums are plain sums in the order of the keys; the merge does not divide.
// dv: the width of a value head; the partial results and the output have dv dims a head.
// The keys are cut into runs of PA_RUN by their absolute position.  One workgroup per (token, query head,
// run): each of its four waves takes 64 keys of the run (lane i scores key i with a full dot product over
// dh from its own cache row; for the value product lane i owns output dims i, i + 64, ...), keeps
// (maximum, normalizer, sums) in float32, the waves are merged through LDS in their order and the workgroup
// leaves one partial result; a second kernel merges the runs in ascending order (the (maximum, normalizer,
// accumulator) merge the reference does across simdgroups, crates/macllm-kernels/src/metal/paged_decode.metal:145-183).
// Which keys meet in a wave, and the order of every sum, depend on the query's position alone: a token's
// result is bit for bit the same whatever else the step holds and however long the longest context is.
#define ATT_MAX_DH 256
#define ATT_WIDE_DH 1024         // rows shared by all heads (latents) may be this wide: a second build of the per-token kernel
#define PA_RUN 256
#define PA_WAVES (PA_RUN / WAVE)

template <typename T, bool FAST_EXP, int MOST = ATT_MAX_DH>
__global__ void __launch_bounds__(PA_RUN)
paged_attention_kernel(const T* __restrict__ q, long q_ld, int Hq, int Hkv, int dh, int dv,
                       const T* __restrict__ k_base, const T* __restrict__ v_base, long page_stride,
                       int page_size, const int* __restrict__ block_tables, int max_pages,
                       const int* __restrict__ lane_of_token, const int* __restrict__ positions, float scale,
                       int window, int kept, const float* __restrict__ slopes, const float* __restrict__ log_bias, int runs,
                       float* __restrict__ partial, const float* __restrict__ head_scales,
                       const float* __restrict__ score_bias, int sigmoid) {
  typedef T vec4 __attribute__((ext_vector_type(4)));
  __shared__ __align__(16) float q_shared[MOST];
  __shared__ float p_shared[PA_WAVES][WAVE];
  __shared__ long row_shared[PA_WAVES][WAVE];     // base of the key's (page, kv head) block of values
  __shared__ int offset_shared[PA_WAVES][WAVE];   // the key's place inside its page
  __shared__ float wave_ml[PA_WAVES][2];
  __shared__ float wave_o[PA_WAVES][MOST];
  const long token = blockIdx.x;
  const int head = blockIdx.y;
  const int run = blockIdx.z;
  const int query_position = positions[token];
  const int first_key = first_visible_key(query_position, window);
  if (((run + 1) * PA_RUN <= first_key && run * PA_RUN >= kept) || run * PA_RUN > query_position) return;   // no key of this run is visible
  const int kvh = head / (Hq / Hkv);
  const int tid = threadIdx.x;
  const int lane = tid & (WAVE - 1);
  const int wave = tid / WAVE;
  const int* table = block_tables + (long)lane_of_token[token] * max_pages;
  const T* q_row = q + token * q_ld + (long)head * dh;
  for (int i = tid; i < dh; i += PA_RUN) q_shared[i] = to_float(q_row[i]);
  __syncthreads();

  const int key = run * PA_RUN + wave * WAVE + lane;
  const bool visible = (key >= first_key || key < kept) && key <= query_position;
  float score = -INFINITY;
  long row_offset = 0;
  int offset = 0;
  if (visible) {
    const int page = table[key / page_size];
    offset = key % page_size;
    row_offset = (long)page * page_stride + (long)kvh * page_size * dv;
    const T* k_row = k_base + (long)page * page_stride + ((long)kvh * page_size + offset) * dh;
    float dot = 0.f;
    if (dh % 4 == 0 && page_stride % 4 == 0 && ((unsigned long long)k_base % (4 * sizeof(T))) == 0) {
      for (int i = 0; i < dh; i += 4) {
        const vec4 piece = *reinterpret_cast<const vec4*>(k_row + i);
#pragma unroll
        for (int j = 0; j < 4; ++j) dot = fmaf(q_shared[i + j], to_float<T>(piece[j]), dot);
      }
    } else {
      for (int i = 0; i < dh; ++i) dot = fmaf(q_shared[i], to_float(k_row[i]), dot);
    }
    score = dot * scale;
    if (head_scales) score *= head_scales[head];
    if (slopes) score = fmaf(-slopes[head], (float)(query_position - key), score);
    if (log_bias) score = fmaf(-log_bias[2 * head], log1pf(log_bias[2 * head + 1] * (float)(query_position - key)), score);
    if (score_bias) score += score_bias[head];
  }
  const float maximum = sigmoid ? 0.f : wave_max(score);    // -inf for a wave without visible keys
  float p = 0.f;
  if (visible) {
    if (sigmoid) p = 1.0f / (1.0f + (FAST_EXP ? __expf(-score) : expf(-score)));
    else p = FAST_EXP ? __expf(score - maximum) : expf(score - maximum);
  }
  p_shared[wave][lane] = p;
  row_shared[wave][lane] = row_offset;
  offset_shared[wave][lane] = offset;
  __syncthreads();
  const int wave_first = run * PA_RUN + wave * WAVE;
  // a wave that holds kept first keys walks from its start: the keys between them and the window weigh 0 and are
  // not added (their cells may be anything)
  const int from = wave_first < kept ? 0 : min(WAVE, max(0, first_key - wave_first));
  const int to = min(WAVE, max(0, query_position - wave_first + 1));
  if (lane == 0) {
    // the normalizer: the probabilities added up in the order of their keys (a sum whose order the keys fix,
    // not the lanes: the tiled kernel below forms the same sum without a pass over the wave)
    float normalizer = 0.f;
    for (int j = from; j < to; ++j) normalizer += p_shared[wave][j];
    wave_ml[wave][0] = maximum;
    wave_ml[wave][1] = normalizer;
  }
#pragma unroll 4
  for (int i = 0; i < MOST / WAVE; ++i) {
    const int dim = lane + i * WAVE;
    if (dim < dv) {
      // sixteen values asked for at once, then added in the order of their keys (one at a time, each load would
      // wait for the one before: 64 round trips a wave); a key past the last reads the last again and is not added
      float sum = 0.f;
      for (int j0 = from; j0 < to; j0 += 16) {
        float values[16];
#pragma unroll
        for (int u = 0; u < 16; ++u) {
          const int j = min(j0 + u, to - 1);
          values[u] = to_float(v_base[row_shared[wave][j] + (long)dim * page_size + offset_shared[wave][j]]);
        }
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int u = 0; u < 16; ++u) {
          const float weight_u = p_shared[wave][min(j0 + u, WAVE - 1)];
          const float added = fmaf(weight_u, values[u], sum);
          sum = (j0 + u < to && (kept <= 0 || weight_u != 0.f)) ? added : sum;
        }
      }
      wave_o[wave][dim] = sum;
    }
  }
  __syncthreads();
  // the waves in their order; a wave without keys has the weight exp(-inf) = 0
  float best = wave_ml[0][0];
#pragma unroll
  for (int w = 1; w < PA_WAVES; ++w) best = fmaxf(best, wave_ml[w][0]);
  float* mine = partial + ((token * Hq + head) * runs + run) * (long)(dv + 2);
  float weight[PA_WAVES];
  float denominator = 0.f;
#pragma unroll
  for (int w = 0; w < PA_WAVES; ++w) {
    weight[w] = FAST_EXP ? __expf(wave_ml[w][0] - best) : expf(wave_ml[w][0] - best);
    denominator = fmaf(weight[w], wave_ml[w][1], denominator);
  }
  if (tid == 0) {
    mine[0] = best;
    mine[1] = denominator;
  }
  for (int dim = tid; dim < dv; dim += PA_RUN) {
    float sum = 0.f;
#pragma unroll
    for (int w = 0; w < PA_WAVES; ++w) sum = fmaf(weight[w], wave_o[w][dim], sum);
    mine[2 + dim] = sum;
  }
}

// The same partial results for steps whose lanes hold several tokens, from a workgroup that takes PT_QUERIES
// consecutive tokens of one lane, one query head and one run of PA_RUN keys: the run's keys and values go through
// LDS once for all of its queries, 64 keys at a time (the per-token kernel above fetches them once a token: a
// prompt of 2,048 tokens reads every key a thousand times).  A query's scores, softmax and sums are the per-token
// kernel's, operation for operation: 64 keys a wave-sized group in the order of their positions, lane i scoring
// key i with a dot product in ascending dims, the group's maximum and normalizer over the wave, lane d summing
// dim d in ascending keys, the four groups of a run weighted and added in their order.  So a position's result is
// the same bits from either kernel: whole prompts, portions and single tokens agree.
// Wave w takes the queries w, w + 4, ... of the tile.
// The largest value of a wave, in every lane: shifts within the rows of 16 lanes, then the last lane of a row
// to the row behind it, then the last lane of the lower half to the upper half (the data-parallel primitives of
// this GPU family; a maximum does not depend on the order it is taken in, so this is wave_max without six trips
// through the LDS crossbar).
template <int CONTROL, int ROW_MASK>
__device__ __forceinline__ float dpp_or_minus_infinity(float x) {
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(__builtin_bit_cast(int, -INFINITY), __builtin_bit_cast(int, x),
                                                               CONTROL, ROW_MASK, 0xf, false));
}

__device__ __forceinline__ float wave_max_dpp(float v) {
  v = fmaxf(v, dpp_or_minus_infinity<0x111, 0xf>(v));      // row_shr:1
  v = fmaxf(v, dpp_or_minus_infinity<0x112, 0xf>(v));      // row_shr:2
  v = fmaxf(v, dpp_or_minus_infinity<0x114, 0xf>(v));      // row_shr:4
  v = fmaxf(v, dpp_or_minus_infinity<0x118, 0xf>(v));      // row_shr:8: lane 15 of each row holds the row's maximum
  v = fmaxf(v, dpp_or_minus_infinity<0x142, 0xa>(v));      // row_bcast:15 into rows 1 and 3
  v = fmaxf(v, dpp_or_minus_infinity<0x143, 0xc>(v));      // row_bcast:31 into rows 2 and 3: lane 63 holds the wave's maximum
  return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), 63));
}

#define PT_QUERIES 16
#define PT_PER_WAVE (PT_QUERIES / PA_WAVES)
#define PT_PAD 4

// DIMS: dims of a head a lane sums (1, 2 or 4: the head size in units of 64, rounded up)
template <typename T, bool FAST_EXP, int DIMS>
__global__ void __launch_bounds__(PA_RUN)
paged_attention_tile_kernel(const T* __restrict__ q, long q_ld, int Hq, int Hkv, int dh, int dv,
                            const T* __restrict__ k_base, const T* __restrict__ v_base, long page_stride,
                            int page_size, const int* __restrict__ block_tables, int max_pages,
                            const int* __restrict__ query_tiles, int tile_tokens, const int* __restrict__ cu_seqlens,
                            const int* __restrict__ positions, float scale, int window, int kept,
                            const float* __restrict__ slopes, const float* __restrict__ log_bias, int runs,
                            float* __restrict__ partial, const float* __restrict__ head_scales,
                            const float* __restrict__ score_bias, int sigmoid) {
  typedef T vec4 __attribute__((ext_vector_type(4)));
  extern __shared__ __align__(16) float tile_lds[];
  const int k_ld = dh + PT_PAD;                      // a key's row in LDS
  const int v_ld = WAVE + PT_PAD;                    // a dim's row of values in LDS
  const int p_ld = WAVE + PT_PAD;                    // a query's row of probabilities in LDS
  float* q_lds = tile_lds;                           // [PT_QUERIES][dh]
  float* k_lds = q_lds + PT_QUERIES * dh;            // [64][k_ld]
  float* v_lds = k_lds + WAVE * k_ld;                // [dv][v_ld]
  float* p_lds = v_lds + dv * v_ld;                  // [PA_WAVES][PT_PER_WAVE][p_ld]
  const int subtiles = tile_tokens / PT_QUERIES;
  const int tile = blockIdx.x / subtiles;
  const int head = blockIdx.y;
  const int run = blockIdx.z;
  const int lane_of_tile = query_tiles[2 * tile];
  if (lane_of_tile < 0) return;                      // a row of the table that holds nothing (a step of fixed capacity)
  const int first_row = query_tiles[2 * tile + 1] + (blockIdx.x - tile * subtiles) * PT_QUERIES;
  const int lane_end = cu_seqlens[lane_of_tile + 1];
  const int tile_end = min(query_tiles[2 * tile + 1] + tile_tokens, lane_end);
  const int count = min(PT_QUERIES, tile_end - first_row);          // queries of this workgroup
  if (count <= 0) return;
  const int last_position = positions[first_row + count - 1];      // positions ascend within a lane
  const int first_position = positions[first_row];
  const int tile_first_key = first_visible_key(first_position, window);     // the oldest key any query of the tile sees
  if (run * PA_RUN > last_position || ((run + 1) * PA_RUN <= tile_first_key && run * PA_RUN >= kept)) return;
  const int kvh = head / (Hq / Hkv);
  const int tid = threadIdx.x;
  const int lane = tid & (WAVE - 1);
  const int wave = tid / WAVE;
  const int* table = block_tables + (long)lane_of_tile * max_pages;
  for (int index = tid; index < count * dh; index += PA_RUN) {
    const int query = index / dh;
    q_lds[index] = to_float(q[(long)(first_row + query) * q_ld + (long)head * dh + (index - query * dh)]);
  }
  // what a wave keeps of its queries' groups: (maximum, normalizer, sums of lane's dims), group by group
  float group_max[PT_PER_WAVE][PA_WAVES], group_norm[PT_PER_WAVE][PA_WAVES], group_o[PT_PER_WAVE][PA_WAVES][DIMS];
#pragma unroll
  for (int i = 0; i < PT_PER_WAVE; ++i)
#pragma unroll
    for (int g = 0; g < PA_WAVES; ++g) {
      group_max[i][g] = -INFINITY;
      group_norm[i][g] = 0.f;
#pragma unroll
      for (int d = 0; d < DIMS; ++d) group_o[i][g][d] = 0.f;
    }
  int query_position[PT_PER_WAVE], query_first[PT_PER_WAVE];
#pragma unroll
  for (int i = 0; i < PT_PER_WAVE; ++i) {
    const int query = wave + i * PA_WAVES;
    query_position[i] = query < count ? positions[first_row + query] : -1;
    query_first[i] = first_visible_key(max(query_position[i], 0), window);
  }

  // one group of 64 keys; called with a constant group so that what a wave keeps of it stays in registers
  auto take_group = [&](auto group_constant) {
    constexpr int g = decltype(group_constant)::value;
    const int group_first = run * PA_RUN + g * WAVE;
    if (group_first > last_position || (group_first + WAVE <= tile_first_key && group_first >= kept)) return;       // the same for every thread
    __syncthreads();                                    // the group before is read (and the queries are laid down)
    // keys group_first .. group_first + 63 that some query of the tile sees; the others (cells never written,
    // pages the request does not hold) are not fetched and lie in LDS as zeros that nobody multiplies
    const int keys = min(WAVE, last_position - group_first + 1);
    const int skipped = max(0, tile_first_key - group_first);      // keys before every query's window: their pages may be gone
    {
      // keys: four threads a key, each a quarter of its dims, 4 dims a load
      const int key_in = tid >> 2;
      const int quarter = dh >> 2;
      const int dim0 = (tid & 3) * quarter;
      float* to = k_lds + key_in * k_ld + dim0;
      if (key_in < keys && (key_in >= skipped || group_first + key_in < kept)) {
        const int key = group_first + key_in;
        const int page = table[key / page_size];
        const T* from = k_base + (long)page * page_stride + ((long)kvh * page_size + key % page_size) * dh + dim0;
        for (int d = 0; d < quarter; d += 4) {
          const vec4 piece = *reinterpret_cast<const vec4*>(from + d);
          *reinterpret_cast<float4*>(to + d) = make_float4(to_float<T>(piece[0]), to_float<T>(piece[1]),
                                                           to_float<T>(piece[2]), to_float<T>(piece[3]));
        }
      } else {
        for (int d = 0; d < quarter; d += 4) *reinterpret_cast<float4*>(to + d) = make_float4(0.f, 0.f, 0.f, 0.f);
      }
    }
    {
      // values: a thread a key (the lanes of a wave walk along a page's tokens), the waves take every fourth dim
      const int key_in = lane;
      if (key_in < keys && (key_in >= skipped || group_first + key_in < kept)) {
        const int key = group_first + key_in;
        const int page = table[key / page_size];
        const T* from = v_base + (long)page * page_stride + (long)kvh * dv * page_size + key % page_size;
        for (int dim = wave; dim < dv; dim += PA_WAVES) v_lds[dim * v_ld + key_in] = to_float(from[(long)dim * page_size]);
      } else {
        for (int dim = wave; dim < dv; dim += PA_WAVES) v_lds[dim * v_ld + key_in] = 0.f;
      }
    }
    __syncthreads();
    // the wave's four queries together: a key's dims and a key's values come out of LDS once for the four (LDS, not
    // the arithmetic, is what this kernel waits for); every query's products and sums are the ones of the per-token
    // kernel in their order.  A query that sees no key of the group ends with what its group started with
    // (maximum -inf, zeros); a query slot past the tile's last is computed on whatever LDS holds and never stored.
    float dot[PT_PER_WAVE];
#pragma unroll
    for (int i = 0; i < PT_PER_WAVE; ++i) dot[i] = 0.f;
    {
      const float* k_row = k_lds + lane * k_ld;
      for (int d = 0; d < dh; d += 4) {
        const float4 kv = *reinterpret_cast<const float4*>(k_row + d);
#pragma unroll
        for (int i = 0; i < PT_PER_WAVE; ++i) {
          const float4 qv = *reinterpret_cast<const float4*>(q_lds + (wave + i * PA_WAVES) * dh + d);
          dot[i] = fmaf(qv.x, kv.x, dot[i]);
          dot[i] = fmaf(qv.y, kv.y, dot[i]);
          dot[i] = fmaf(qv.z, kv.z, dot[i]);
          dot[i] = fmaf(qv.w, kv.w, dot[i]);
        }
      }
    }
    float* p_rows = p_lds + wave * (PT_PER_WAVE * p_ld);          // this wave's four rows of probabilities: no barrier, the wave runs in step
#pragma unroll
    for (int i = 0; i < PT_PER_WAVE; ++i) {
      const int position = query_position[i];
      const int first_key = query_first[i];
      const int key = group_first + lane;
      const bool visible = (key >= first_key || key < kept) && key <= position;
      float score = -INFINITY;
      if (visible) {
        score = dot[i] * scale;
        if (head_scales) score *= head_scales[head];
        if (slopes) score = fmaf(-slopes[head], (float)(position - key), score);
        if (log_bias) score = fmaf(-log_bias[2 * head], log1pf(log_bias[2 * head + 1] * (float)(position - key)), score);
        if (score_bias) score += score_bias[head];
      }
      const float maximum = sigmoid ? 0.f : wave_max_dpp(score);
      float p = 0.f;
      if (visible) {
        if (sigmoid) p = 1.0f / (1.0f + (FAST_EXP ? __expf(-score) : expf(-score)));
        else p = FAST_EXP ? __expf(score - maximum) : expf(score - maximum);
      }
      p_rows[i * p_ld + lane] = p;
      group_max[i][g] = maximum;
    }
    __builtin_amdgcn_wave_barrier();
    // sums over all 64 keys of the group: a key the query does not see has the probability 0 and a finite
    // value (a key some query of the tile sees, or a zero laid down above), so it adds an exact zero and the
    // sums are those of the keys from `from` to `to` in their order, which is what the per-token kernel adds
    {
      float sums[PT_PER_WAVE][DIMS];
#pragma unroll
      for (int i = 0; i < PT_PER_WAVE; ++i)
#pragma unroll
        for (int d = 0; d < DIMS; ++d) sums[i][d] = 0.f;
      const float* v_row[DIMS];
#pragma unroll
      for (int d = 0; d < DIMS; ++d) v_row[d] = v_lds + min(lane + d * WAVE, dv - 1) * v_ld;
      // the normalizers: lane i adds the probabilities of query i in the order of the keys
      const float* p_mine = p_rows + (lane & (PT_PER_WAVE - 1)) * p_ld;
      float normalizer = 0.f;
#pragma unroll
      for (int j = 0; j < WAVE; j += 4) {
        const float4 mine = *reinterpret_cast<const float4*>(p_mine + j);
        normalizer += mine.x;
        normalizer += mine.y;
        normalizer += mine.z;
        normalizer += mine.w;
        float4 pj[PT_PER_WAVE];
#pragma unroll
        for (int i = 0; i < PT_PER_WAVE; ++i) pj[i] = *reinterpret_cast<const float4*>(p_rows + i * p_ld + j);
#pragma unroll
        for (int d = 0; d < DIMS; ++d) {
          if (d * WAVE < dv) {                          // the same for every lane
            const float4 vj = *reinterpret_cast<const float4*>(v_row[d] + j);
#pragma unroll
            for (int i = 0; i < PT_PER_WAVE; ++i) {
              sums[i][d] = fmaf(pj[i].x, vj.x, sums[i][d]);
              sums[i][d] = fmaf(pj[i].y, vj.y, sums[i][d]);
              sums[i][d] = fmaf(pj[i].z, vj.z, sums[i][d]);
              sums[i][d] = fmaf(pj[i].w, vj.w, sums[i][d]);
            }
          }
        }
      }
#pragma unroll
      for (int i = 0; i < PT_PER_WAVE; ++i) {
        group_norm[i][g] = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, normalizer), i));
#pragma unroll
        for (int d = 0; d < DIMS; ++d) group_o[i][g][d] = sums[i][d];
      }
    }
    __builtin_amdgcn_wave_barrier();
  };
  take_group(std::integral_constant<int, 0>{});
  take_group(std::integral_constant<int, 1>{});
  take_group(std::integral_constant<int, 2>{});
  take_group(std::integral_constant<int, 3>{});
  static_assert(PA_WAVES == 4, "a run of keys is four groups of 64");
  // the groups of the run in their order, as the per-token kernel merges its waves
#pragma unroll
  for (int i = 0; i < PT_PER_WAVE; ++i) {
    const int position = query_position[i];
    const int first_key = query_first[i];
    if (position < 0 || ((run + 1) * PA_RUN <= first_key && run * PA_RUN >= kept) || run * PA_RUN > position) continue;    // the per-token kernel writes nothing either
    float best = group_max[i][0];
#pragma unroll
    for (int g = 1; g < PA_WAVES; ++g) best = fmaxf(best, group_max[i][g]);
    float weight[PA_WAVES];
    float denominator = 0.f;
#pragma unroll
    for (int g = 0; g < PA_WAVES; ++g) {
      weight[g] = FAST_EXP ? __expf(group_max[i][g] - best) : expf(group_max[i][g] - best);
      denominator = fmaf(weight[g], group_norm[i][g], denominator);
    }
    const long token = first_row + wave + i * PA_WAVES;
    float* mine = partial + ((token * Hq + head) * runs + run) * (long)(dv + 2);
    if (lane == 0) {
      mine[0] = best;
      mine[1] = denominator;
    }
#pragma unroll
    for (int d = 0; d < DIMS; ++d) {
      const int dim = lane + d * WAVE;
      if (dim < dv) {
        float sum = 0.f;
#pragma unroll
        for (int g = 0; g < PA_WAVES; ++g) sum = fmaf(weight[g], group_o[i][g][d], sum);
        mine[2 + dim] = sum;
      }
    }
  }
}

template <typename T, bool FAST_EXP>
__global__ void paged_attention_merge_kernel(const float* __restrict__ partial, int Hq, int dh, int runs,
                                             const int* __restrict__ positions, int window, int kept,
                                             const float* __restrict__ sinks, float fixed_sink, int has_fixed_sink,
                                             T* __restrict__ out, long out_ld, int sigmoid, const T* __restrict__ gate,
                                             long gate_ld) {
  const long token = blockIdx.x;
  const int head = blockIdx.y;
  const int query_position = positions[token];
  const int first_key = first_visible_key(query_position, window);
  const int first_run = first_key / PA_RUN;
  // a caller's bound on the contexts sizes the work area: a token beyond that bound merges the runs that
  // were launched for it and never reads outside the area
  const int last_run = min(query_position / PA_RUN, runs - 1);
  const float* theirs = partial + ((token * Hq + head) * runs) * (long)(dh + 2);
  for (int dim = threadIdx.x; dim < dh; dim += blockDim.x) {
    float maximum = -INFINITY, denominator = 0.f, sum = 0.f;
    for (int run = 0; run <= last_run; ++run) {
      if (run < first_run && run * PA_RUN >= kept) continue;       // behind the window and past the kept first keys: never written
      const float* one = theirs + (long)run * (dh + 2);
      const float larger = fmaxf(maximum, one[0]);
      const float keep = FAST_EXP ? __expf(maximum - larger) : expf(maximum - larger);     // 0 the first time
      const float weight = FAST_EXP ? __expf(one[0] - larger) : expf(one[0] - larger);
      denominator = denominator * keep + weight * one[1];
      sum = sum * keep + weight * one[2 + dim];
      maximum = larger;
    }
    if (sinks || has_fixed_sink) {
      // the sink: a term of the denominator that brings no value
      const float sink = sinks ? sinks[head] : fixed_sink;
      const float larger = fmaxf(maximum, sink);
      const float keep = FAST_EXP ? __expf(maximum - larger) : expf(maximum - larger);
      denominator = denominator * keep + (FAST_EXP ? __expf(sink - larger) : expf(sink - larger));
      sum *= keep;
    }
    const float gated = (sigmoid ? sum : sum / denominator) * output_gate(gate, gate_ld, token, (long)head * dh + dim);
    out[token * out_ld + (long)head * dh + dim] = from_float<T>(gated);
  }
}

// partial: work area of at least T * Hq * runs * (dh + 2) floats, runs = ceil(max_seq_len / PA_RUN), where
// max_seq_len bounds the number of keys (position + 1) of every token of the step.
extern "C" long mi_paged_attention_workspace(int T, int Hq, int dh, int max_seq_len) {
  if (T <= 0 || Hq <= 0 || dh <= 0 || max_seq_len <= 0) return 0;
  return (long)T * Hq * ((max_seq_len + PA_RUN - 1) / PA_RUN) * (dh + 2);
}

// LDS of a workgroup of the tiled kernel: the tile's queries, 64 keys, their values, a wave's probabilities
static size_t paged_attention_tile_lds(int dh, int dv) {
  return ((size_t)PT_QUERIES * dh + (size_t)WAVE * (dh + PT_PAD) + (size_t)dv * (WAVE + PT_PAD) +
          (size_t)PT_QUERIES * (WAVE + PT_PAD)) * sizeof(float);
}

template <typename T, bool FAST_EXP, int DIMS>
static int raise_tile_lds(size_t bytes) {
  // beyond 64 KiB a kernel has to be told once per device that it may have that much (gfx950 has 160 KiB)
  static size_t raised[64] = {};        // per instantiation of this function: the most it was told so far
  int device = 0;
  if (hipGetDevice(&device) != hipSuccess || device < 0 || device >= 64) return ERR_BAD_ARGUMENT;
  if (raised[device] >= bytes) return 0;
  if (hipFuncSetAttribute((const void*)paged_attention_tile_kernel<T, FAST_EXP, DIMS>, hipFuncAttributeMaxDynamicSharedMemorySize,
                          (int)bytes) != hipSuccess) {
    (void)hipGetLastError();
    return ERR_UNSUPPORTED_SIZE;
  }
  raised[device] = bytes;
  return 0;
}

// query_tiles (optional) [num_tiles, 2] = (lane or -1, first token row) of runs of up to tile_tokens tokens of one
// lane (tile_tokens a multiple of 16), with cu_seqlens [lanes + 1]: the step's lanes hold several tokens, and the
// partial results come from the kernel that shares a run's keys among the queries of a tile (the same bits).
// dv: the width of a value head (the work area is sized for it: mi_paged_attention_workspace(T, Hq, dv, ...));
// log_bias, sinks: see above.
extern "C" int mi_paged_attention(const void* q, int dtype, long q_ld, int T, int Hq, int Hkv, int dh, int dv,
                                  const void* k_base, const void* v_base, long page_stride, int page_size,
                                  const int* block_tables, int max_pages, const int* lane_of_token,
                                  const int* positions, float scale, int window, int kept, const float* slopes,
                                  const float* log_bias, const float* sinks, float fixed_sink, int has_fixed_sink,
                                  int max_seq_len, float* partial, long partial_floats, void* out, long out_ld,
                                  const int* query_tiles, int num_tiles, int tile_tokens, const int* cu_seqlens,
                                  const float* head_scales, const float* score_bias, int sigmoid, const void* gate,
                                  long gate_ld, hipStream_t stream) {
  if (gate && gate_ld < (long)Hq * dv) return ERR_BAD_ARGUMENT;
  if ((score_bias && !sigmoid) || (sigmoid && (sinks || has_fixed_sink)) || (sinks && has_fixed_sink)) return ERR_BAD_ARGUMENT;
  if (kept < 0 || (kept > 0 && window <= 0)) return ERR_BAD_ARGUMENT;
  if (T <= 0 || Hq <= 0 || Hkv <= 0 || Hq % Hkv != 0 || dh <= 0 || dv <= 0 || page_size <= 0 || max_pages <= 0 ||
      max_seq_len <= 0 || !partial)
    return ERR_BAD_ARGUMENT;
  if (dh > ATT_WIDE_DH || dv > ATT_WIDE_DH) return ERR_UNSUPPORTED_SIZE;
  const bool wide = dh > ATT_MAX_DH || dv > ATT_MAX_DH;
  const int runs = (max_seq_len + PA_RUN - 1) / PA_RUN;
  if (Hq > 65535 || runs > 65535) return ERR_UNSUPPORTED_SIZE;
  if (partial_floats < mi_paged_attention_workspace(T, Hq, dv, max_seq_len)) return ERR_BAD_ARGUMENT;
  const int element = dtype == DT_F32 ? 4 : 2;
  // the tiled kernel: head sizes in steps of 16, 4 elements a load from the cache
  bool tiled = query_tiles != nullptr && num_tiles > 0 && cu_seqlens != nullptr && tile_tokens > 0 &&
               tile_tokens % PT_QUERIES == 0 && dh % 16 == 0 && dv <= ATT_MAX_DH && page_stride % 4 == 0 &&
               ((uintptr_t)k_base % (4 * element)) == 0 && (long)num_tiles * (tile_tokens / PT_QUERIES) <= 0x7fffffffL;
  const size_t tile_lds = paged_attention_tile_lds(dh, dv);
  const int dims = dv <= WAVE ? 1 : dv <= 2 * WAVE ? 2 : 4;
  if (tiled && tile_lds > 64 * 1024) {
    int code;
    if (dtype == DT_F32)
      code = dims == 1 ? raise_tile_lds<float, false, 1>(tile_lds)
                       : dims == 2 ? raise_tile_lds<float, false, 2>(tile_lds) : raise_tile_lds<float, false, 4>(tile_lds);
    else
      code = dims == 1 ? raise_tile_lds<bf16_t, true, 1>(tile_lds)
                       : dims == 2 ? raise_tile_lds<bf16_t, true, 2>(tile_lds) : raise_tile_lds<bf16_t, true, 4>(tile_lds);
    if (code != 0) tiled = false;                      // the per-token kernel takes any size
  }
  const dim3 grid(T, Hq, runs);
  const dim3 tile_grid(tiled ? num_tiles * (tile_tokens / PT_QUERIES) : 1, Hq, runs);
  const dim3 merge_grid(T, Hq);
  const int merge_threads = dv <= WAVE ? WAVE : dv <= 2 * WAVE ? 2 * WAVE : 4 * WAVE;
  if (dtype == DT_F32) {
#define TILE_LAUNCH(T_, FAST_, DIMS_)                                                                                 \
  paged_attention_tile_kernel<T_, FAST_, DIMS_><<<tile_grid, PA_RUN, tile_lds, stream>>>(                              \
      (const T_*)q, q_ld, Hq, Hkv, dh, dv, (const T_*)k_base, (const T_*)v_base, page_stride, page_size, block_tables, \
      max_pages, query_tiles, tile_tokens, cu_seqlens, positions, scale, window, kept, slopes, log_bias, runs, partial, \
      head_scales, score_bias, sigmoid)
    if (tiled && dims == 1) TILE_LAUNCH(float, false, 1);
    else if (tiled && dims == 2) TILE_LAUNCH(float, false, 2);
    else if (tiled) TILE_LAUNCH(float, false, 4);
    else
{
      if (wide)
        paged_attention_kernel<float, false, ATT_WIDE_DH><<<grid, PA_RUN, 0, stream>>>(
            (const float*)q, q_ld, Hq, Hkv, dh, dv, (const float*)k_base, (const float*)v_base, page_stride, page_size,
            block_tables, max_pages, lane_of_token, positions, scale, window, kept, slopes, log_bias, runs, partial,
            head_scales, score_bias, sigmoid);
      else
        paged_attention_kernel<float, false><<<grid, PA_RUN, 0, stream>>>(
            (const float*)q, q_ld, Hq, Hkv, dh, dv, (const float*)k_base, (const float*)v_base, page_stride, page_size,
            block_tables, max_pages, lane_of_token, positions, scale, window, kept, slopes, log_bias, runs, partial,
            head_scales, score_bias, sigmoid);
    }
    RETURN_IF_LAUNCH_FAILED();
    paged_attention_merge_kernel<float, false><<<merge_grid, merge_threads, 0, stream>>>(
        partial, Hq, dv, runs, positions, window, kept, sinks, fixed_sink, has_fixed_sink, (float*)out, out_ld, sigmoid,
        (const float*)gate, gate_ld);
  } else if (dtype == DT_BF16) {
    if (tiled && dims == 1) TILE_LAUNCH(bf16_t, true, 1);
    else if (tiled && dims == 2) TILE_LAUNCH(bf16_t, true, 2);
    else if (tiled) TILE_LAUNCH(bf16_t, true, 4);
    else
{
      if (wide)
        paged_attention_kernel<bf16_t, true, ATT_WIDE_DH><<<grid, PA_RUN, 0, stream>>>(
            (const bf16_t*)q, q_ld, Hq, Hkv, dh, dv, (const bf16_t*)k_base, (const bf16_t*)v_base, page_stride,
            page_size, block_tables, max_pages, lane_of_token, positions, scale, window, kept, slopes, log_bias, runs,
            partial, head_scales, score_bias, sigmoid);
      else
        paged_attention_kernel<bf16_t, true><<<grid, PA_RUN, 0, stream>>>(
            (const bf16_t*)q, q_ld, Hq, Hkv, dh, dv, (const bf16_t*)k_base, (const bf16_t*)v_base, page_stride,
            page_size, block_tables, max_pages, lane_of_token, positions, scale, window, kept, slopes, log_bias, runs,
            partial, head_scales, score_bias, sigmoid);
    }
    RETURN_IF_LAUNCH_FAILED();
    paged_attention_merge_kernel<bf16_t, true><<<merge_grid, merge_threads, 0, stream>>>(
        partial, Hq, dv, runs, positions, window, kept, sinks, fixed_sink, has_fixed_sink, (bf16_t*)out, out_ld, sigmoid,
        (const bf16_t*)gate, gate_ld);
  } else {
    return ERR_BAD_ARGUMENT;
  }
#undef TILE_LAUNCH
  RETURN_IF_LAUNCH_FAILED();
  return 0;
}

// ---------------------------------------------------------------- decode attention, split over the context
// For batches of single-token queries in bfloat16.  grid = (splits, kv heads, tokens); a block
// takes one page-aligned range of `split_keys` keys of one request and one kv head and serves
// all G query heads of that kv head from the same K and V loads:
//   scores : LPR = DH/8 lanes share a key row (16 B each), partial dots are summed across them;
//   softmax: over the block's range in float32 (scores staged in LDS), giving (max, sum);
//   values : V pages are [dim, token]; lane d owns output dim d and reads 8 tokens per load.
// Every block writes an unnormalized partial output with its (max, sum); the merge kernel
// combines the splits (the same (maximum, normalizer, accumulator) merge the reference does
// across simdgroups, crates/macllm-kernels/src/metal/paged_decode.metal:145-183).
#define DEC_THREADS 256
#define DEC_WAVES (DEC_THREADS / WAVE)
#define DEC_MAX_SPLIT 512
#define DEC_AHEAD 4               // rounds of keys asked for at once
#define DEC_MERGE_SPLITS 256     // splits whose factors the merge keeps in LDS

struct alignas(16) bf16x8 {
  bf16_t v[8];
};

// dv: the width of a value head and of a head's output (any width; the keys' when it is DH).  head_scales
// (a multiplier on a head's scores, after `scale`), score_bias and slopes (score -= slopes[head] * distance) may be null.
// dh: the width of a key head, a multiple of 8 up to DH (the lanes of a key's row past it bring nothing).  sigmoid: a visible key weighs
// sigmoid(score + score_bias[head]) on its own; the block then records (0, 1) as its (max, sum) and the merge adds
// the partial outputs as they are.  Dynamic LDS: DEC_WAVES * G * dv floats.
// kept > 0 (with a window): the keys at positions below kept stay visible; those that lie before the window's first
// page are the work of one more block, blockIdx.x == splits, whose partial result stands behind the others'
// (an empty one, maximum -inf, when the window still reaches them).
template <int DH, int G>
__global__ void __launch_bounds__(DEC_THREADS)
decode_attention_kernel(const bf16_t* __restrict__ q, long q_ld, int Hq, const bf16_t* __restrict__ k_base,
                        const bf16_t* __restrict__ v_base, long page_stride, int page_size,
                        const int* __restrict__ block_tables, int max_pages,
                        const int* __restrict__ lane_of_token, const int* __restrict__ positions, float scale,
                        int window, int split_keys, int splits, float* __restrict__ partial_o,
                        float* __restrict__ partial_ml, int dh, int dv, const float* __restrict__ head_scales,
                        const float* __restrict__ score_bias, const float* __restrict__ slopes, int sigmoid, int kept) {
  constexpr int LPR = DH / 8;
  constexpr int KPW = WAVE / LPR;
  constexpr int KPB = KPW * DEC_WAVES;
  __shared__ float s_lds[G][DEC_MAX_SPLIT];
  __shared__ float red[DEC_WAVES][G];
  extern __shared__ float acc_lds[];             // [DEC_WAVES][G][dv]

  const int split = blockIdx.x;
  const int kvh = blockIdx.y;
  const long token = blockIdx.z;
  const int pos = positions[token];
  const int first_key = first_visible_key(pos, window);
  const int first_page_key = (first_key / page_size) * page_size;
  const bool kept_block = split == splits;                   // only launched with kept > 0
  const int stride = kept > 0 ? splits + 1 : splits;         // partial results of a head
  const int range_lo = kept_block ? 0 : first_page_key + split * split_keys;
  if (range_lo > pos) return;
  const int range_hi = kept_block ? min(kept, first_page_key) : min(range_lo + split_keys, pos + 1);
  const int count = range_hi - range_lo;
  const int tid = threadIdx.x;
  if (count <= 0) {          // the kept first keys are inside the window's pages: nothing of their own
    for (int index = tid; index < G * dv; index += DEC_THREADS)
      partial_o[((token * Hq + kvh * G + index / dv) * stride + split) * dv + index % dv] = 0.f;
    if (tid < G) {
      float* ml = partial_ml + ((token * Hq + kvh * G + tid) * stride + split) * 2;
      ml[0] = sigmoid ? 0.f : -INFINITY;
      ml[1] = sigmoid ? 1.f : 0.f;
    }
    return;
  }
  const int* table = block_tables + (long)lane_of_token[token] * max_pages;
  const int lane = tid & (WAVE - 1);
  const int wave = tid / WAVE;
  const int r = lane / LPR;
  const int c = lane % LPR;

  float qf[G][8];
  float offset_of[G], slope_of[G];
  const bool brings = c * 8 < dh;                // whether this lane's piece of a key's row exists
#pragma unroll
  for (int g = 0; g < G; ++g) {
    const float factor = head_scales ? scale * head_scales[kvh * G + g] : scale;
    offset_of[g] = score_bias ? score_bias[kvh * G + g] : 0.f;
    slope_of[g] = slopes ? slopes[kvh * G + g] : 0.f;
    bf16x8 packed;
    if (brings) {
      packed = *reinterpret_cast<const bf16x8*>(q + token * q_ld + (long)(kvh * G + g) * dh + c * 8);
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j) packed.v[j] = (bf16_t)0.f;
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) qf[g][j] = (float)packed.v[j] * factor;
  }

  // scores, DEC_AHEAD rounds of keys at a time: their page ids, then their rows, are asked for together
  for (int base0 = 0; base0 < count; base0 += DEC_AHEAD * KPB) {
    int key[DEC_AHEAD], page[DEC_AHEAD];
    bf16x8 packed[DEC_AHEAD];
#pragma unroll
    for (int a = 0; a < DEC_AHEAD; ++a) {
      key[a] = range_lo + min(base0 + a * KPB + wave * KPW + r, count - 1);      // (past the range: its last key again, dropped below)
      page[a] = table[key[a] / page_size];
    }
#pragma unroll
    for (int a = 0; a < DEC_AHEAD; ++a)
      packed[a] = *reinterpret_cast<const bf16x8*>(k_base + (long)page[a] * page_stride +
                                                   ((long)kvh * page_size + key[a] % page_size) * dh + (brings ? c * 8 : 0));
#pragma unroll
    for (int a = 0; a < DEC_AHEAD; ++a) {
      const int local = base0 + a * KPB + wave * KPW + r;
      if (base0 + a * KPB >= count) break;                                       // the same for every lane
      float s[G], kf[8];
#pragma unroll
      for (int j = 0; j < 8; ++j) kf[j] = brings ? (float)packed[a].v[j] : 0.f;
#pragma unroll
      for (int g = 0; g < G; ++g) {
        s[g] = 0.f;
#pragma unroll
        for (int j = 0; j < 8; ++j) s[g] = fmaf(qf[g][j], kf[j], s[g]);
      }
#pragma unroll
      for (int offset = LPR / 2; offset > 0; offset >>= 1)
#pragma unroll
        for (int g = 0; g < G; ++g) s[g] += __shfl_xor(s[g], offset, WAVE);
      if (local < count && c == 0) {
#pragma unroll
        for (int g = 0; g < G; ++g) {
          const float score = fmaf(-slope_of[g], (float)(pos - key[a]), s[g] + offset_of[g]);
          s_lds[g][local] = (key[a] >= first_key || key[a] < kept) ? score : -INFINITY;
        }
      }
    }
  }
  __syncthreads();

  float m[G], l[G];
  if (sigmoid) {
    // every key on its own: 1 / (1 + exp(-s)); a key before the window's first (-inf) weighs nothing
#pragma unroll
    for (int g = 0; g < G; ++g) {
      for (int i = tid; i < count; i += DEC_THREADS) {
        const float score = s_lds[g][i];
        s_lds[g][i] = score == -INFINITY ? 0.f : __builtin_amdgcn_rcpf(1.f + __expf(-score));
      }
      m[g] = 0.f;
      l[g] = 1.f;
    }
  } else {
    // softmax over the range: maximum, then exp and sum
#pragma unroll
    for (int g = 0; g < G; ++g) {
      float v = -INFINITY;
      for (int i = tid; i < count; i += DEC_THREADS) v = fmaxf(v, s_lds[g][i]);
      v = wave_max(v);
      if (lane == 0) red[wave][g] = v;
    }
    __syncthreads();
#pragma unroll
    for (int g = 0; g < G; ++g) {
      float v = red[0][g];
#pragma unroll
      for (int w = 1; w < DEC_WAVES; ++w) v = fmaxf(v, red[w][g]);
      m[g] = v;
    }
    __syncthreads();
#pragma unroll
    for (int g = 0; g < G; ++g) {
      float sum = 0.f;
      for (int i = tid; i < count; i += DEC_THREADS) {
        const float p = m[g] == -INFINITY ? 0.f : __expf(s_lds[g][i] - m[g]);
        s_lds[g][i] = p;
        sum += p;
      }
      sum = wave_sum(sum);
      if (lane == 0) red[wave][g] = sum;
    }
    __syncthreads();
#pragma unroll
    for (int g = 0; g < G; ++g) {
      float v = 0.f;
#pragma unroll
      for (int w = 0; w < DEC_WAVES; ++w) v += red[w][g];
      l[g] = v;
    }
  }
  __syncthreads();

  // values: each wave takes every fourth page of the range, 64 dims of the value head at a time
  const int range_pages = (count + page_size - 1) / page_size;
  for (int dim0 = 0; dim0 < dv; dim0 += WAVE) {
    const int dim = dim0 + lane;
    float acc[G];
#pragma unroll
    for (int g = 0; g < G; ++g) acc[g] = 0.f;
    if (dim < dv) {
      for (int pg = wave; pg < range_pages; pg += DEC_WAVES) {
        const int local0 = pg * page_size;
        const int page = table[(range_lo + local0) / page_size];
        const int keys_here = min(page_size, count - local0);
        const bf16_t* v_row = v_base + (long)page * page_stride + ((long)kvh * dv + dim) * page_size;
        for (int j0 = 0; j0 < keys_here; j0 += 8) {
          const bf16x8 packed = *reinterpret_cast<const bf16x8*>(v_row + j0);
#pragma unroll
          for (int j = 0; j < 8; ++j) {
            if (j0 + j < keys_here) {
              const float value = (float)packed.v[j];
#pragma unroll
              for (int g = 0; g < G; ++g) acc[g] = fmaf(s_lds[g][local0 + j0 + j], value, acc[g]);
            }
          }
        }
      }
#pragma unroll
      for (int g = 0; g < G; ++g) acc_lds[((long)wave * G + g) * dv + dim] = acc[g];
    }
  }
  __syncthreads();
  for (int index = tid; index < G * dv; index += DEC_THREADS) {
    const int g = index / dv;
    const int dim = index - g * dv;
    float sum = 0.f;
#pragma unroll
    for (int w = 0; w < DEC_WAVES; ++w) sum += acc_lds[((long)w * G + g) * dv + dim];
    partial_o[((token * Hq + kvh * G + g) * stride + split) * dv + dim] = sum;
  }
  if (tid < G) {
    float* ml = partial_ml + ((token * Hq + kvh * G + tid) * stride + split) * 2;
    ml[0] = m[tid];
    ml[1] = l[tid];
  }
}

// out[token, head, :] = sum_s exp(m_s - M) o_s / sum_s exp(m_s - M) l_s over the splits that hold keys
// (dh: the width of a head's output); sigmoid: the plain sum of the splits' outputs.
__global__ void decode_merge_kernel(const float* __restrict__ partial_o, const float* __restrict__ partial_ml,
                                    const int* __restrict__ positions, int window, int page_size,
                                    int split_keys, int splits, int Hq, int dh, bf16_t* __restrict__ out,
                                    long out_ld, int sigmoid, int kept, const float* __restrict__ sinks,
                                    const bf16_t* __restrict__ gate, long gate_ld) {
  const long token = blockIdx.x;
  const int head = blockIdx.y;
  const int pos = positions[token];
  const int first_key = first_visible_key(pos, window);
  const int first_page_key = (first_key / page_size) * page_size;
  const int used = min(splits, (pos - first_page_key) / split_keys + 1);
  const int stride = kept > 0 ? splits + 1 : splits;
  const float* ml = partial_ml + (token * Hq + head) * stride * 2;
  const float* o = partial_o + (token * Hq + head) * (long)stride * dh;
  if (sigmoid) {
    for (int dim = threadIdx.x; dim < dh; dim += blockDim.x) {
      float sum = 0.f;
      for (int s = 0; s < used; ++s) sum += o[(long)s * dh + dim];
      if (kept > 0) sum += o[(long)splits * dh + dim];
      out[token * out_ld + (long)head * dh + dim] = (bf16_t)(sum * output_gate(gate, gate_ld, token, (long)head * dh + dim));
    }
    return;
  }
  if (kept > 0 || sinks) {
    // the block of the kept first keys and a sink (a term of the denominator that brings no value) beside the splits
    const float sink = sinks ? sinks[head] : -INFINITY;
    float maximum = sink;
    for (int s = 0; s < used; ++s) maximum = fmaxf(maximum, ml[2 * s]);
    if (kept > 0) maximum = fmaxf(maximum, ml[2 * splits]);
    float denominator = sinks ? __expf(sink - maximum) : 0.f;
    for (int s = 0; s < used; ++s) denominator += __expf(ml[2 * s] - maximum) * ml[2 * s + 1];
    const float kept_factor = kept > 0 ? __expf(ml[2 * splits] - maximum) : 0.f;
    if (kept > 0) denominator += kept_factor * ml[2 * splits + 1];
    for (int dim = threadIdx.x; dim < dh; dim += blockDim.x) {
      float sum = 0.f;
      for (int s = 0; s < used; ++s) sum += __expf(ml[2 * s] - maximum) * o[(long)s * dh + dim];
      if (kept > 0) sum += kept_factor * o[(long)splits * dh + dim];
      out[token * out_ld + (long)head * dh + dim] = (bf16_t)(sum / denominator * output_gate(gate, gate_ld, token, (long)head * dh + dim));
    }
    return;
  }
  // the splits' factors exp(m_s - M) and the denominator, by the first wave (a split a lane at a time), through LDS
  // for all; more splits than the table holds: every thread forms them for itself
  __shared__ float factor_lds[DEC_MERGE_SPLITS];
  __shared__ float denominator_lds;
  if (used <= DEC_MERGE_SPLITS) {
    if (threadIdx.x < WAVE) {
      float maximum = -INFINITY;
      for (int s = threadIdx.x; s < used; s += WAVE) maximum = fmaxf(maximum, ml[2 * s]);
      maximum = wave_max(maximum);
      float denominator = 0.f;
      for (int s = threadIdx.x; s < used; s += WAVE) {
        const float factor = __expf(ml[2 * s] - maximum);
        factor_lds[s] = factor;
        denominator += factor * ml[2 * s + 1];
      }
      denominator = wave_sum(denominator);
      if (threadIdx.x == 0) denominator_lds = denominator;
    }
    __syncthreads();
    const float denominator = denominator_lds;
    for (int dim = threadIdx.x; dim < dh; dim += blockDim.x) {
      float sum = 0.f;
      for (int s = 0; s < used; ++s) sum = fmaf(factor_lds[s], o[(long)s * dh + dim], sum);
      out[token * out_ld + (long)head * dh + dim] = (bf16_t)(sum / denominator * output_gate(gate, gate_ld, token, (long)head * dh + dim));
    }
    return;
  }
  float maximum = -INFINITY;
  for (int s = 0; s < used; ++s) maximum = fmaxf(maximum, ml[2 * s]);
  float denominator = 0.f;
  for (int s = 0; s < used; ++s) denominator += __expf(ml[2 * s] - maximum) * ml[2 * s + 1];
  for (int dim = threadIdx.x; dim < dh; dim += blockDim.x) {
    float sum = 0.f;
    for (int s = 0; s < used; ++s) sum += __expf(ml[2 * s] - maximum) * o[(long)s * dh + dim];
    out[token * out_ld + (long)head * dh + dim] = (bf16_t)(sum / denominator * output_gate(gate, gate_ld, token, (long)head * dh + dim));
  }
}

template <int DH, int G>
static int launch_decode(const bf16_t* q, long q_ld, int T, int Hq, int Hkv, const bf16_t* k_base,
                         const bf16_t* v_base, long page_stride, int page_size, const int* block_tables,
                         int max_pages, const int* lane_of_token, const int* positions, float scale, int window,
                         int split_keys, int splits, float* partial_o, float* partial_ml, int dh, int dv,
                         const float* head_scales, const float* score_bias, const float* slopes, int sigmoid, int kept,
                         hipStream_t stream) {
  const dim3 grid(kept > 0 ? splits + 1 : splits, Hkv, T);
  const size_t dynamic = sizeof(float) * DEC_WAVES * G * (size_t)dv;
  decode_attention_kernel<DH, G><<<grid, DEC_THREADS, dynamic, stream>>>(
      q, q_ld, Hq, k_base, v_base, page_stride, page_size, block_tables, max_pages, lane_of_token, positions,
      scale, window, split_keys, splits, partial_o, partial_ml, dh, dv, head_scales, score_bias, slopes, sigmoid, kept);
  return 0;
}

// Returns ERR_UNSUPPORTED_SIZE for shapes this kernel does not cover (the caller then uses
// mi_paged_attention): head_dim a multiple of 8 up to 128, 1..8 query heads per kv head, page_size a multiple of 8,
// split_keys a multiple of page_size and at most DEC_MAX_SPLIT, values of up to 256 dims a head.
// partial_o holds T * Hq * splits * dv floats (with kept > 0: splits + 1 a head, and partial_ml likewise).
// kept (with a window): the first keys that stay visible, at most DEC_MAX_SPLIT; sinks (float32 per query head, or
// null): exp(sink) is one more term of the softmax's denominator.
extern "C" int mi_decode_attention_forms(const void* q, long q_ld, int T, int Hq, int Hkv, int dh, int dv,
                                         const void* k_base, const void* v_base, long page_stride, int page_size,
                                         const int* block_tables, int max_pages, const int* lane_of_token,
                                         const int* positions, float scale, int window, int split_keys, int splits,
                                         float* partial_o, float* partial_ml, void* out, long out_ld,
                                         const float* head_scales, const float* score_bias, const float* slopes,
                                         int sigmoid, int kept, const float* sinks, const void* gate, long gate_ld,
                                         hipStream_t stream) {
  if (T <= 0 || Hq <= 0 || Hkv <= 0 || Hq % Hkv != 0 || page_size <= 0 || splits <= 0 || max_pages <= 0 || dv <= 0)
    return ERR_BAD_ARGUMENT;
  if (kept < 0 || (kept > 0 && window <= 0) || (sinks && sigmoid)) return ERR_BAD_ARGUMENT;
  if (gate && gate_ld < (long)Hq * dv) return ERR_BAD_ARGUMENT;
  if (kept > DEC_MAX_SPLIT) return ERR_UNSUPPORTED_SIZE;
  const int G = Hq / Hkv;
  if (dh <= 0 || dh % 8 != 0 || dh > 128 || G > 8 || page_size % 8 != 0 || split_keys % page_size != 0 ||
      split_keys <= 0 || split_keys > DEC_MAX_SPLIT || T > 65535 || Hkv > 65535 || dv > 256)
    return ERR_UNSUPPORTED_SIZE;
  if (score_bias != nullptr && !sigmoid) return ERR_BAD_ARGUMENT;
  const int lanes_width = dh <= 64 ? 64 : 128;
#define DECODE_CASE(DH_, G_)                                                                                     \
  if (lanes_width == DH_ && G == G_)                                                                                      \
    launch_decode<DH_, G_>((const bf16_t*)q, q_ld, T, Hq, Hkv, (const bf16_t*)k_base, (const bf16_t*)v_base,     \
                           page_stride, page_size, block_tables, max_pages, lane_of_token, positions, scale,     \
                           window, split_keys, splits, partial_o, partial_ml, dh, dv, head_scales, score_bias,   \
                           slopes, sigmoid, kept, stream);
  DECODE_CASE(64, 1) DECODE_CASE(64, 2) DECODE_CASE(64, 3) DECODE_CASE(64, 4) DECODE_CASE(64, 5)
  DECODE_CASE(64, 6) DECODE_CASE(64, 7) DECODE_CASE(64, 8)
  DECODE_CASE(128, 1) DECODE_CASE(128, 2) DECODE_CASE(128, 3) DECODE_CASE(128, 4) DECODE_CASE(128, 5)
  DECODE_CASE(128, 6) DECODE_CASE(128, 7) DECODE_CASE(128, 8)
#undef DECODE_CASE
  RETURN_IF_LAUNCH_FAILED();
  const dim3 merge_grid(T, Hq);
  const int merge_threads = dv <= 64 ? 64 : dv <= 128 ? 128 : 256;
  decode_merge_kernel<<<merge_grid, merge_threads, 0, stream>>>(partial_o, partial_ml, positions, window, page_size,
                                                                split_keys, splits, Hq, dv, (bf16_t*)out, out_ld,
                                                                sigmoid, kept, sinks, (const bf16_t*)gate, gate_ld);
  RETURN_IF_LAUNCH_FAILED();
  return 0;
}

// The ordinary form: softmax weights, values as wide as the keys.
extern "C" int mi_decode_attention(const void* q, long q_ld, int T, int Hq, int Hkv, int dh, const void* k_base,
                                   const void* v_base, long page_stride, int page_size, const int* block_tables,
                                   int max_pages, const int* lane_of_token, const int* positions, float scale,
                                   int window, int split_keys, int splits, float* partial_o, float* partial_ml,
                                   void* out, long out_ld, hipStream_t stream) {
  return mi_decode_attention_forms(q, q_ld, T, Hq, Hkv, dh, dh, k_base, v_base, page_stride, page_size, block_tables,
                                   max_pages, lane_of_token, positions, scale, window, split_keys, splits, partial_o,
                                   partial_ml, out, out_ld, nullptr, nullptr, nullptr, 0, 0, nullptr, nullptr, 0, stream);
}

// ---------------------------------------------------------------- decode attention without a workspace argument
// The partial results live in an array of the library's device image (see static_scratch.h).  In host code
// the array's name is a stand-in, not a device address: its address on each GPU is asked for once per
// device, with that device current, and kept.
#include "static_scratch.h"
#include <mutex>

static __device__ __align__(256) float scratch[MI_STATIC_SCRATCH_BYTES / sizeof(float)];

#define STATIC_MAX_DEVICES 64
static float* scratch_of_device[STATIC_MAX_DEVICES];
static std::mutex scratch_lock;

// The address of this GPU's copy of `scratch`, or null with *error set.
static float* static_scratch(hipError_t* error) {
  int device = -1;
  *error = hipGetDevice(&device);
  if (*error != hipSuccess) return nullptr;
  if (device < 0 || device >= STATIC_MAX_DEVICES) {
    *error = hipErrorInvalidDevice;
    return nullptr;
  }
  std::lock_guard<std::mutex> guard(scratch_lock);
  if (scratch_of_device[device] == nullptr) {
    float* address = nullptr;
    *error = hipGetSymbolAddress((void**)&address, HIP_SYMBOL(scratch));
    if (*error != hipSuccess) return nullptr;
    scratch_of_device[device] = address;
  }
  return scratch_of_device[device];
}

extern "C" long mi_static_scratch_bytes(void) { return (long)MI_STATIC_SCRATCH_BYTES; }

extern "C" int mi_decode_attention_static(const void* q, long q_ld, int T, int Hq, int Hkv, int dh,
                                          const void* k_base, const void* v_base, long page_stride, int page_size,
                                          const int* block_tables, int max_pages, const int* lane_of_token,
                                          const int* positions, float scale, int window, int split_keys,
                                          int splits, void* out, long out_ld, hipStream_t stream) {
  if (T <= 0 || Hq <= 0 || dh <= 0 || splits <= 0) return ERR_BAD_ARGUMENT;
  // partial outputs first, their (max, sum) behind them, each part in whole runs of 256 bytes
  const unsigned long long rows = (unsigned long long)T * (unsigned long long)Hq * (unsigned long long)splits;
  const unsigned long long o_floats = (rows * (unsigned long long)dh + 63ull) & ~63ull;
  const unsigned long long ml_floats = (rows * 2ull + 63ull) & ~63ull;
  if (o_floats + ml_floats > MI_STATIC_SCRATCH_BYTES / sizeof(float)) return ERR_UNSUPPORTED_SIZE;
  hipError_t error = hipSuccess;
  float* base = static_scratch(&error);
  if (base == nullptr) return (int)error;
  return mi_decode_attention(q, q_ld, T, Hq, Hkv, dh, k_base, v_base, page_stride, page_size, block_tables,
                             max_pages, lane_of_token, positions, scale, window, split_keys, splits, base,
                             base + o_floats, out, out_ld, stream);
}

#include "attn_prefill.h"

// The widths the values are computed with when they are not the keys' (the cached width rounded up to one of them),
// and the query heads that share a key fragment at that width: the accumulators of a set grow with it.
static int padded_value_width(int dv) {
  const int widths[] = {32, 64, 96, 128, 160, 192, 256};
  for (int width : widths)
    if (dv <= width) return width;
  return 0;
}

// The same kernel for two further forms (bfloat16, head_dim 64 or 128):
//   values of another width than the keys (dv a multiple of 4 up to 256; softmax, no window bias or sink), and
//   sigmoid weights with a multiplier and a bias per head (either null), values as wide as the keys.
// Returns ERR_UNSUPPORTED_SIZE for what it does not cover (the caller uses mi_paged_attention).
extern "C" int mi_prefill_attention_forms(const void* q, long q_ld, int Hq, int Hkv, int dh, int dv, const void* k_base,
                                          const void* v_base, long page_stride, int page_size,
                                          const int* block_tables, int max_pages, const int* tiles, int n_tiles,
                                          const int* cu_seqlens, const int* start_pos, float scale, int window,
                                          int max_seq_len, void* out, long out_ld, int sigmoid,
                                          const float* head_scales, const float* score_bias, hipStream_t stream) {
  if (n_tiles <= 0 || Hq <= 0 || Hkv <= 0 || Hq % Hkv != 0 || page_size <= 0 || max_pages <= 0 || dv <= 0)
    return ERR_BAD_ARGUMENT;
  const int G = Hq / Hkv;
  if ((dh != 64 && dh != 128) || page_size % 4 != 0 || q_ld % 8 != 0 || out_ld % 4 != 0 || Hkv > 65535 || G > 64 ||
      dv % 4 != 0 || n_tiles > (1 << 28))
    return ERR_UNSUPPORTED_SIZE;
  if (sigmoid ? dv != dh : (dv == dh || head_scales || score_bias)) return ERR_UNSUPPORTED_SIZE;
  const int width = sigmoid ? dh : padded_value_width(dv);
  if (width == 0) return ERR_UNSUPPORTED_SIZE;
  const int widest = width > dh ? width : dh;
  int most = widest <= 64 ? 4 : widest <= 128 ? 2 : 1;
  if (most > 2 && max_seq_len <= 2048 && 4L * n_tiles * Hkv * ((G + most - 1) / most) < PREFILL_FILL_BLOCKS) most = 2;
  const int passes = (G + most - 1) / most;
  const int nset = (G + passes - 1) / passes;
  const dim3 grid(4 * n_tiles, Hkv, passes);
#define FORM_ARGS                                                                                              \
  (const bf16_t*)q, q_ld, Hq, Hkv, (const bf16_t*)k_base, (const bf16_t*)v_base, page_stride, page_size,       \
      block_tables, max_pages, tiles, cu_seqlens, start_pos, scale, window, (bf16_t*)out, out_ld, nullptr,     \
      nullptr, dv, head_scales, score_bias
#define SIGMOID_CASE(DH_, NSET_)                                                                               \
  if (sigmoid && dh == DH_ && nset == NSET_)                                                                   \
    prefill_attention_kernel<DH_, NSET_, BIAS_NONE, DH_, true, false><<<grid, PREFILL_WAVES * WAVE, 0, stream>>>(FORM_ARGS);
#define PADDED_CASE(DH_, DV_, NSET_)                                                                           \
  if (!sigmoid && dh == DH_ && width == DV_ && nset == NSET_)                                                  \
    prefill_attention_kernel<DH_, NSET_, BIAS_NONE, DV_, false, true><<<grid, PREFILL_WAVES * WAVE, 0, stream>>>(FORM_ARGS);
  SIGMOID_CASE(64, 1) SIGMOID_CASE(64, 2) SIGMOID_CASE(64, 3) SIGMOID_CASE(64, 4)
  SIGMOID_CASE(128, 1) SIGMOID_CASE(128, 2)
  PADDED_CASE(64, 32, 1) PADDED_CASE(64, 32, 2) PADDED_CASE(64, 32, 3) PADDED_CASE(64, 32, 4)
  PADDED_CASE(64, 64, 1) PADDED_CASE(64, 64, 2) PADDED_CASE(64, 64, 3) PADDED_CASE(64, 64, 4)
  PADDED_CASE(64, 96, 1) PADDED_CASE(64, 96, 2) PADDED_CASE(64, 128, 1) PADDED_CASE(64, 128, 2)
  PADDED_CASE(64, 160, 1) PADDED_CASE(64, 192, 1) PADDED_CASE(64, 256, 1)
  PADDED_CASE(128, 32, 1) PADDED_CASE(128, 32, 2) PADDED_CASE(128, 64, 1) PADDED_CASE(128, 64, 2)
  PADDED_CASE(128, 96, 1) PADDED_CASE(128, 96, 2) PADDED_CASE(128, 128, 1) PADDED_CASE(128, 128, 2)
  PADDED_CASE(128, 160, 1) PADDED_CASE(128, 192, 1) PADDED_CASE(128, 256, 1)
#undef SIGMOID_CASE
#undef PADDED_CASE
#undef FORM_ARGS
  RETURN_IF_LAUNCH_FAILED();
  return 0;
}

// tiles: int32 [n_tiles, 2] = (lane, first token row of the tile); a tile never crosses a lane.
// Returns ERR_UNSUPPORTED_SIZE for shapes it does not cover (the caller uses mi_paged_attention).
extern "C" int mi_prefill_attention(const void* q, long q_ld, int Hq, int Hkv, int dh, const void* k_base,
                                    const void* v_base, long page_stride, int page_size, const int* block_tables,
                                    int max_pages, const int* tiles, int n_tiles, const int* cu_seqlens,
                                    const int* start_pos, float scale, int window, int max_seq_len, void* out,
                                    long out_ld, const float* log_bias, const float* sinks, int kept,
                                    const float* slopes, const void* gate, long gate_ld, hipStream_t stream) {
  if ((log_bias && slopes) || (gate && (gate_ld < (long)Hq * dh || gate_ld % 4 != 0 || (uintptr_t)gate % 8 != 0)))
    return ERR_BAD_ARGUMENT;
  if (n_tiles <= 0 || Hq <= 0 || Hkv <= 0 || Hq % Hkv != 0 || page_size <= 0 || max_pages <= 0)
    return ERR_BAD_ARGUMENT;
  if (kept < 0 || (kept > 0 && window <= 0)) return ERR_BAD_ARGUMENT;      // first keys are kept behind a window
  const int G = Hq / Hkv;
  if ((dh != 64 && dh != 128) || page_size % 4 != 0 || q_ld % 8 != 0 || out_ld % 4 != 0 || Hkv > 65535 || G > 64)
    return ERR_UNSUPPORTED_SIZE;
  // up to four query heads share every K and V fragment; head size 128 holds twice the registers per head, and
  // more than two heads would spill.  A grid that would leave compute units with fewer than two workgroups, over
  // contexts of up to 2,048 keys (max_seq_len: an upper bound of the step's longest context, 0 = not known), is
  // bound by the softmax arithmetic of its longest tiles: it takes sets of two heads, so that twice the
  // workgroups, every other pass from the light end, spread that work.  Over longer contexts the keys and
  // values that four heads share count for more (a 2,048-token portion of the 0.5B shape behind 2,048 tokens
  // of context: 7.29 ms with two heads a set, 6.85 with four; behind 30,000 tokens 19.0 and 16.4).
  int most = dh == 128 ? 2 : 4;
  if (most > 2 && max_seq_len <= 2048 && 4L * n_tiles * Hkv * ((G + most - 1) / most) < PREFILL_FILL_BLOCKS) most = 2;
  const int passes = (G + most - 1) / most;
  const int nset = (G + passes - 1) / passes;
  if (n_tiles > (1 << 28)) return ERR_UNSUPPORTED_SIZE;
  const dim3 grid(4 * n_tiles, Hkv, passes);
#define PREFILL_LAUNCH(DH_, NSET_, BIAS_)                                                                      \
  prefill_attention_kernel<DH_, NSET_, BIAS_><<<grid, PREFILL_WAVES * WAVE, 0, stream>>>(                     \
      (const bf16_t*)q, q_ld, Hq, Hkv, (const bf16_t*)k_base, (const bf16_t*)v_base, page_stride, page_size,  \
      block_tables, max_pages, tiles, cu_seqlens, start_pos, scale, window, (bf16_t*)out, out_ld, log_bias, sinks, \
      DH_, nullptr, nullptr, kept, slopes, (const bf16_t*)gate, gate_ld)
#define PREFILL_CASE(DH_, NSET_)                                                                              \
  if (dh == DH_ && nset == NSET_) {                                                                           \
    if (log_bias) PREFILL_LAUNCH(DH_, NSET_, BIAS_LOG);                                                       \
    else if (slopes) PREFILL_LAUNCH(DH_, NSET_, BIAS_LINEAR);                                                 \
    else PREFILL_LAUNCH(DH_, NSET_, BIAS_NONE);                                                               \
  }
  PREFILL_CASE(64, 1) PREFILL_CASE(64, 2) PREFILL_CASE(64, 3) PREFILL_CASE(64, 4)
  PREFILL_CASE(128, 1) PREFILL_CASE(128, 2)
#undef PREFILL_LAUNCH
#undef PREFILL_CASE
  RETURN_IF_LAUNCH_FAILED();
  return 0;
}
