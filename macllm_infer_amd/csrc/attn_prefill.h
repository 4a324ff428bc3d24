// Prefill attention on the matrix cores: bfloat16, head_dim 64 or 128 (padded: any multiple of 8 up to 128).
// grid = (4 x query tiles, kv heads, head passes): a tile is up to 64 consecutive tokens of one lane and a
// workgroup takes 16 of them with the query heads of one kv
// head (NSET column sets that share every K and V fragment).  The keys, from the first visible
// one to the workgroup's last position, are split in eight runs of whole 32-key steps, one per
// wave, read straight from the cache pages (the portion's own keys were written by rope_kv_store
// before), four steps in flight at a time; the eight partial results are merged through LDS,
// set by set.  Workgroups with the longest contexts (the last tiles) are launched first, in every
// other head pass last.
#pragma once
#include "attn_mfma.h"

#define PREFILL_STEPS 4
#define PREFILL_WAVES 8
#define PREFILL_FILL_BLOCKS 512   // two workgroups for each of the 256 compute units

// BIAS: BIAS_LOG, the scores lose log_bias[head] = (r1, r2) -> r1 * ln(1 + r2 * distance); BIAS_LINEAR, they lose
// slopes[head] * distance.  sinks (may be null): one more term exp(sinks[head]) of the softmax's denominator.
// DV: the width the values are computed with, the keys' or, PADDED, the next width of the launch's table above
// value_dim, the width of the cached values and of a head's output (a multiple of 4).
// SIGMOID: a visible key weighs sigmoid(score * scale * head_scales[head] + score_bias[head]) on its own (either
// pointer may be null: 1 and 0); no maximum, no normalizer, the waves' partial sums are added as they are.
// PADDED_KEYS: the cached keys and the queries are
// key_dim wide, a multiple of 8 and at most DH.  out_gate: see output_gate (softmax weights; rows in pieces of four).
template <int DH, int NSET, int BIAS = BIAS_NONE, int DV = DH, bool SIGMOID = false, bool PADDED = false,
          bool PADDED_KEYS = false>
__global__ void __launch_bounds__(PREFILL_WAVES * WAVE)
prefill_attention_kernel(const bf16_t* __restrict__ q, long q_ld, int Hq, int Hkv, const bf16_t* __restrict__ k_base,
                         const bf16_t* __restrict__ v_base, long page_stride, int page_size,
                         const int* __restrict__ block_tables, int max_pages, const int* __restrict__ tiles,
                         const int* __restrict__ cu_seqlens, const int* __restrict__ start_pos, float scale,
                         int window, bf16_t* __restrict__ out, long out_ld,
                         const float* __restrict__ log_bias = nullptr, const float* __restrict__ sinks = nullptr,
                         int value_dim = DV, const float* __restrict__ head_scales = nullptr,
                         const float* __restrict__ score_bias = nullptr, int kept = 0,
                         const float* __restrict__ slopes = nullptr, const bf16_t* __restrict__ out_gate = nullptr,
                         long gate_ld = 0, int key_dim = DH) {
  constexpr int ITEMS = 2 + 4 * (DV / 16);                    // m, l and the accumulator of one set
  __shared__ float part[PREFILL_WAVES][ITEMS][WAVE];
  __shared__ int wave_pages[PREFILL_WAVES][WAVE];
  // heavy ones first; every other head pass the other way round, so that workgroups of two passes that
  // run side by side bring about the same work together
  const int block = (blockIdx.z & 1) ? blockIdx.x : gridDim.x - 1 - blockIdx.x;
  const int tile = block / 4;
  const int kvh = blockIdx.y;
  const int G = Hq / Hkv;
  const int head0 = kvh * G + blockIdx.z * NSET;             // first head of this pass
  const int request = tiles[2 * tile];
  if (request < 0) return;                                    // a row of the table past the step's own runs
  const int lane = threadIdx.x & (WAVE - 1);
  const int wave = threadIdx.x / WAVE;
  const int qd = lane / 16;
  const int n = lane % 16;
  const int lane_end = cu_seqlens[request + 1];
  const int first_token = tiles[2 * tile + 1] + 16 * (block % 4);
  if (first_token >= lane_end) return;                        // the whole workgroup
  const int token = first_token + n;
  const bool has_query = token < lane_end;
  const int base_position = start_pos[request] - cu_seqlens[request];
  const int position = base_position + token;
  const int last_position = base_position + min(first_token + 15, lane_end - 1);
  const int first_position = base_position + first_token;
  // every column of the wave holds a query (16 tokens, and the head sets divide the heads): the wave's bounds are known
  const bool full_tile = first_token + 16 <= lane_end && (blockIdx.z + 1) * NSET <= G;

  mfma_bf16x8 q_frag[NSET][DH / 32];
  int col_pos[NSET];
#pragma unroll
  for (int s = 0; s < NSET; ++s) {
    const bool valid = has_query && blockIdx.z * NSET + s < G;
    col_pos[s] = valid ? position : -1;
#pragma unroll
    for (int kk = 0; kk < DH / 32; ++kk) {
      if (valid && (!PADDED_KEYS || 32 * kk + 8 * qd < key_dim)) {
        q_frag[s][kk] = *reinterpret_cast<const mfma_bf16x8*>(q + (long)token * q_ld +
                                                               (long)(head0 + s) * (PADDED_KEYS ? key_dim : DH) +
                                                               32 * kk + 8 * qd);
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j) q_frag[s][kk][j] = (bf16_t)0.f;
      }
    }
  }
  AttnAccumulator<DH, NSET, DV> acc;
  acc.clear();
  AttnGate<NSET> gate;
  if (SIGMOID) {
#pragma unroll
    for (int s = 0; s < NSET; ++s) {
      const int head = min(head0 + s, Hq - 1);
      gate.scale[s] = scale * (head_scales ? head_scales[head] : 1.f);
      gate.bias[s] = score_bias ? score_bias[head] : 0.f;
    }
  }
  AttnBias<NSET> bias;
#pragma unroll
  for (int s = 0; s < NSET; ++s) {
    const int head = min(head0 + s, Hq - 1);
    bias.slope[s] = BIAS == BIAS_LINEAR ? slopes[head] * 1.4426950408889634f : 0.f;
    bias.r1[s] = BIAS == BIAS_LOG ? log_bias[2 * head] : 0.f;
    bias.r2[s] = BIAS == BIAS_LOG ? log_bias[2 * head + 1] : 0.f;
  }
  AttnCache cache;
  cache.k_base = k_base;
  cache.v_base = v_base;
  cache.page_stride = page_stride;
  cache.page_size = page_size;
  cache.kvh = kvh;
  cache.value_dim = value_dim;
  cache.key_dim = key_dim;
  const int* cache_pages = block_tables + (long)request * max_pages;
  const int key_lo = (first_visible_key(first_position, window) / 32) * 32;
  const int key_hi = last_position + 1;
  const int steps = (key_hi - key_lo + 31) / 32;
  const int steps_per_wave = (steps + PREFILL_WAVES - 1) / PREFILL_WAVES;
  const int my_lo = key_lo + 32 * steps_per_wave * wave;
  const int my_hi = min(key_hi, my_lo + 32 * steps_per_wave);
  // the page ids of the run go through LDS, 64 pages at a time (a wave's own corner of it: no
  // barrier), so that a K or V load does not wait for a load of its page id
  auto walk = [&](int from, int to) {
    for (int part_lo = from; part_lo < to;) {
      const int first_page = part_lo / page_size;
      const int part_hi = min(to, (first_page + WAVE) * page_size);
      wave_pages[wave][lane] = cache_pages[min(first_page + lane, max_pages - 1)];
      cache.pages = wave_pages[wave];
      cache.base_page = first_page;
      attend_keys<DH, NSET, PREFILL_STEPS, false, BIAS, DV, SIGMOID, PADDED, PADDED_KEYS>(
          acc, q_frag, col_pos, window, scale, part_lo, part_hi, cache, full_tile ? first_position : -1, last_position,
          bias, &gate, kept);
      part_lo = part_hi;
    }
  };
  walk(my_lo, my_hi);
  // the kept first keys that lie before the window's first step: the last wave, whose own run is the shortest
  if (kept > 0 && key_lo > 0 && wave == PREFILL_WAVES - 1) walk(0, min(kept, key_lo));

  // merge: set s is finished by wave s
#pragma unroll
  for (int s = 0; s < NSET; ++s) {
    // the gate of the outputs this wave will write, asked for ahead of the exchange through LDS
    mfma_bf16x4 gate_piece[DV / 16];
    const bool gated = !SIGMOID && out_gate && wave == s % PREFILL_WAVES && col_pos[s] >= 0;
    if (gated) {
      const bf16_t* gate_row = out_gate + (long)token * gate_ld + (long)(head0 + s) * value_dim;
#pragma unroll
      for (int dt = 0; dt < DV / 16; ++dt)
        if (!PADDED || 16 * dt + 4 * qd < value_dim) gate_piece[dt] = *reinterpret_cast<const mfma_bf16x4*>(gate_row + 16 * dt + 4 * qd);
    }
    __syncthreads();
    part[wave][0][lane] = acc.m[s];
    part[wave][1][lane] = acc.l[s];
#pragma unroll
    for (int dt = 0; dt < DV / 16; ++dt)
#pragma unroll
      for (int i = 0; i < 4; ++i) part[wave][2 + 4 * dt + i][lane] = acc.o[s][dt][i];
    __syncthreads();
    if (wave != s % PREFILL_WAVES) continue;
    if (SIGMOID) {
      if (col_pos[s] < 0) continue;
      bf16_t* o = out + (long)token * out_ld + (long)(head0 + s) * value_dim;
#pragma unroll
      for (int dt = 0; dt < DV / 16; ++dt) {
        mfma_bf16x4 packed;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          float value = 0.f;
#pragma unroll
          for (int w = 0; w < PREFILL_WAVES; ++w) value += part[w][2 + 4 * dt + i][lane];
          packed[i] = (bf16_t)value;
        }
        if (!PADDED || 16 * dt + 4 * qd < value_dim) *reinterpret_cast<mfma_bf16x4*>(o + 16 * dt + 4 * qd) = packed;
      }
      continue;
    }
    float m = -INFINITY;
#pragma unroll
    for (int w = 0; w < PREFILL_WAVES; ++w) m = fmaxf(m, part[w][0][lane]);
    // the sink, in the scores' units of log2: it may be the largest term
    const float sink = sinks ? sinks[min(head0 + s, Hq - 1)] * 1.4426950408889634f : -INFINITY;
    m = fmaxf(m, sink);
    float factor[PREFILL_WAVES];
    float l = 0.f;
#pragma unroll
    for (int w = 0; w < PREFILL_WAVES; ++w) {
      const float m_w = part[w][0][lane];
      factor[w] = m_w == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m_w - m);
      l += part[w][1][lane] * factor[w];
    }
    l += __shfl_xor(l, 16, WAVE);
    l += __shfl_xor(l, 32, WAVE);
    if (sinks) l += __builtin_amdgcn_exp2f(sink - m);       // once for the column: no key, no value
    if (col_pos[s] < 0) continue;
    const float inverse = 1.f / l;
    bf16_t* o = out + (long)token * out_ld + (long)(head0 + s) * value_dim;
#pragma unroll
    for (int dt = 0; dt < DV / 16; ++dt) {
      if (PADDED && 16 * dt + 4 * qd >= value_dim) continue;
      float value[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        value[i] = 0.f;
#pragma unroll
        for (int w = 0; w < PREFILL_WAVES; ++w) value[i] += part[w][2 + 4 * dt + i][lane] * factor[w];
        value[i] *= inverse;
      }
      if (gated) {
#pragma unroll
        for (int i = 0; i < 4; ++i) value[i] *= __frcp_rn(1.0f + __expf(-(float)gate_piece[dt][i]));
      }
      mfma_bf16x4 packed;
#pragma unroll
      for (int i = 0; i < 4; ++i) packed[i] = (bf16_t)value[i];
      *reinterpret_cast<mfma_bf16x4*>(o + 16 * dt + 4 * qd) = packed;
    }
  }
}
