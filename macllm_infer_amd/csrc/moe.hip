// A feed-forward of many small experts of which a token uses a few.
//
//   moe_route        float32 router logits -> softmax, correction, the token's experts and their weights (one wave
//                    a token), and the sigmoid of the shared expert's gate logit; or (mode 1) logits + bias -> the
//                    largest ones and the softmax over those alone; groups of neighbouring experts may restrict
//                    the choice to the best groups
//   moe_plan         the step's (token, choice) rows grouped by expert, every expert's rows starting a tile of 16
//                    places: built on the device by one workgroup, so that no count has to travel to the host and
//                    the launches that follow depend on the number of tokens alone
//   moe_expert_gemm  the grouped product on the matrix cores: a tile's rows (gathered from the tokens' rows, or
//                    the places themselves) with its expert's matrix; epilogue: plain, or the clamped gated
//                    activation of a gate tile and an up tile
//   moe_combine      a token's weighted sum over its choices, in their order, plus the (gated) shared expert
//
// The router may have more outputs than there are experts with matrices: the last ones are identity experts, whose
// output is the token's own row.  The plan gives their choices no place, the sum takes the row itself.
//
// A row of a tile is summed on its own (a column of the matrix cores' result), so a token's numbers do not depend
// on which other rows share its tile or on the place it was given.
#include "mfma_tile.h"

#define MOE_MAX_EXPERTS 1024
#define MOE_PER_LANE (MOE_MAX_EXPERTS / WAVE)

// ---------------------------------------------------------------- router
// The largest number of a wave and the smallest, in every lane: shifts within the rows of 16 lanes, then across them
// (data-parallel primitives: no trips through the LDS crossbar; neither depends on the order it is taken in).
template <int CONTROL, int ROW_MASK>
__device__ __forceinline__ int moved_or(int x, int otherwise) {
  return __builtin_amdgcn_update_dpp(otherwise, x, CONTROL, ROW_MASK, 0xf, false);
}
__device__ __forceinline__ float wave_most(float v) {
  const int none = __builtin_bit_cast(int, -INFINITY);
#define MOST_STEP(C_, M_) v = fmaxf(v, __builtin_bit_cast(float, moved_or<C_, M_>(__builtin_bit_cast(int, v), none)))
  MOST_STEP(0x111, 0xf); MOST_STEP(0x112, 0xf); MOST_STEP(0x114, 0xf); MOST_STEP(0x118, 0xf); MOST_STEP(0x142, 0xa); MOST_STEP(0x143, 0xc);
#undef MOST_STEP
  return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), 63));
}
__device__ __forceinline__ int wave_least(int v) {
#define LEAST_STEP(C_, M_) v = min(v, moved_or<C_, M_>(v, 0x7fffffff))
  LEAST_STEP(0x111, 0xf); LEAST_STEP(0x112, 0xf); LEAST_STEP(0x114, 0xf); LEAST_STEP(0x118, 0xf); LEAST_STEP(0x142, 0xa); LEAST_STEP(0x143, 0xc);
#undef LEAST_STEP
  return __builtin_amdgcn_readlane(v, 63);
}

struct RouteArgs {
  const float* logits;
  long ld;
  int T, E, top;
  const float* correction;
  float scale, eps;
  int mode, renormalize, groups, kept_groups;
  int* chosen;
  float* weights;
  float* gate;
};

// One wave routes one token.  PER_LANE: the most experts a lane holds.
template <int PER_LANE>
__device__ __forceinline__ void route_token(const RouteArgs& a, int token) {
  const int lane = threadIdx.x & (WAVE - 1);
  const int E = a.E, top = a.top;
  const float* row = a.logits + (long)token * a.ld;
  float score[PER_LANE], choice[PER_LANE];
  const int held = (E + WAVE - 1) / WAVE;          // experts a lane holds: the loops below end there (the same in every lane)
  float most = -INFINITY;
#pragma unroll
  for (int j = 0; j < PER_LANE; ++j) {
    if (j >= held) break;
    const int e = lane + WAVE * j;
    score[j] = e < E ? row[e] : -INFINITY;
    choice[j] = (a.correction && e < E) ? a.correction[e] : 0.f;     // (asked for beside the logits)
    most = fmaxf(most, score[j]);
  }
  if (a.mode == 0) {
    most = wave_most(most);
    float total = 0.f;
#pragma unroll
    for (int j = 0; j < PER_LANE; ++j) {
      if (j >= held) break;
      const int e = lane + WAVE * j;
      score[j] = e < E ? expf(score[j] - most) : 0.f;
      total += score[j];
    }
    total = wave_sum(total);
#pragma unroll
    for (int j = 0; j < PER_LANE; ++j) {
      if (j >= held) break;
      const int e = lane + WAVE * j;
      score[j] = score[j] / total;
      choice[j] = e < E ? score[j] + choice[j] : -INFINITY;
    }
  } else if (a.mode == 2) {
    // every output on its own: s = sigmoid(z).  Without a correction the logits decide, whose order is that of the s
#pragma unroll
    for (int j = 0; j < PER_LANE; ++j) {
      if (j >= held) break;
      const int e = lane + WAVE * j;
      const float logit = score[j];
      score[j] = e < E ? 1.0f / (1.0f + expf(-logit)) : 0.f;
      choice[j] = e < E ? (a.correction ? score[j] + choice[j] : logit) : -INFINITY;
    }
  } else {
    // the logits with their bias are what is chosen by and what is weighted
#pragma unroll
    for (int j = 0; j < PER_LANE; ++j) {
      if (j >= held) break;
      const int e = lane + WAVE * j;
      score[j] = e < E ? score[j] + choice[j] : -INFINITY;
      choice[j] = score[j];
    }
  }
  // the expert with the largest number among those whose bit is not set in `out`: ties go to the lower expert
  auto best_of = [&](unsigned out) {
    float best = -INFINITY;
    int best_id = 0x7fffffff;
#pragma unroll
    for (int j = 0; j < PER_LANE; ++j) {
      if (j >= held) break;
      const int e = lane + WAVE * j;
      if (e < E && !(out >> j & 1) && (choice[j] > best || (choice[j] == best && e < best_id))) {
        best = choice[j];
        best_id = e;
      }
    }
    const float largest = wave_most(best);
    return wave_least(best == largest ? best_id : 0x7fffffff);
  };
  if (a.groups > 0) {
    // the best groups, one round each: the largest choice score outside the groups kept so far is its group's score.
    // Everything outside the kept groups ends at minus infinity.
    const int group_size = E / a.groups;
    unsigned kept = 0;                 // bit j: this lane's j-th expert belongs to a kept group
    for (int k = 0; k < a.kept_groups; ++k) {
      const int group = best_of(kept) / group_size;
#pragma unroll
      for (int j = 0; j < PER_LANE; ++j) {
        if (j >= held) break;
        if ((lane + WAVE * j) / group_size == group) kept |= 1u << j;
      }
    }
#pragma unroll
    for (int j = 0; j < PER_LANE; ++j)
      if (j < held && !(kept >> j & 1)) choice[j] = -INFINITY;
  }
  float first_picked = 0.f;        // mode 1: the largest chosen logit, which is the first one picked
  float picked_sum = 0.f;
  float mine = 0.f;            // lane k keeps the score of the k-th choice
  int mine_id = 0;
  for (int k = 0; k < top; ++k) {
    const int best_id = min(best_of(0), E - 1);     // scores that are no numbers pick nothing: whatever is chosen is an expert
    float own = 0.f;
#pragma unroll
    for (int j = 0; j < PER_LANE; ++j)
      if (j < held && lane + WAVE * j == best_id) {
        choice[j] = -INFINITY;
        own = score[j];
      }
    float best_score = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, own), best_id & (WAVE - 1)));
    if (a.mode == 1) {
      if (k == 0) first_picked = best_score;
      best_score = expf(best_score - first_picked);
    }
    picked_sum += best_score;
    if ((k & (WAVE - 1)) == lane) {
      mine = best_score;
      mine_id = best_id;
    }
    if (top > WAVE && lane == 0) {       // more choices than lanes: written as they come
      a.chosen[(long)token * top + k] = best_id;
      a.weights[(long)token * top + k] = best_score;      // divided below
    }
  }
  const float denominator = a.renormalize ? picked_sum + a.eps : 1.0f;
  if (top <= WAVE) {
    if (lane < top) {
      a.chosen[(long)token * top + lane] = mine_id;
      a.weights[(long)token * top + lane] = mine / denominator * a.scale;
    }
  } else if (lane == 0) {
    for (int k = 0; k < top; ++k) a.weights[(long)token * top + k] = a.weights[(long)token * top + k] / denominator * a.scale;
  }
  if (a.gate && lane == 0) a.gate[token] = 1.0f / (1.0f + expf(-row[E]));
}

template <int PER_LANE>
__global__ void __launch_bounds__(256) moe_route_kernel(RouteArgs a) {
  const int token = blockIdx.x * (blockDim.x / WAVE) + threadIdx.x / WAVE;
  if (token < a.T) route_token<PER_LANE>(a, token);
}

static int check_route(const RouteArgs& a) {
  if (!a.logits || !a.chosen || !a.weights || a.T <= 0 || a.E <= 0 || a.top <= 0 || a.top > a.E || a.ld < a.E + (a.gate ? 1 : 0))
    return ERR_BAD_ARGUMENT;
  if (a.E > MOE_MAX_EXPERTS) return ERR_UNSUPPORTED_SIZE;
  if (a.mode < 0 || a.mode > 2) return ERR_BAD_ARGUMENT;
  if (a.mode == 1 && (!a.renormalize || a.groups != 0)) return ERR_BAD_ARGUMENT;
  if (a.groups < 0 || (a.groups > 0 && (a.E % a.groups != 0 || a.kept_groups <= 0 || a.kept_groups > a.groups ||
                                        a.kept_groups * (a.E / a.groups) < a.top)))
    return ERR_BAD_ARGUMENT;
  return 0;
}

// mode 0: softmax over all experts, choice by score + correction, weights score / (sum of the chosen + eps) * scale,
// or without `renormalize` score * scale.  groups > 0 (mode 0): E / groups neighbouring experts form a group, its score
// is its largest score + correction, and only experts of the `kept_groups` best groups can be chosen.
// mode 1: choice by logit + correction (a bias), weights the softmax over the chosen (logit + correction) * scale.
// mode 2: as mode 0 with the sigmoid of each logit in place of the softmax.  correction may be null (nothing is added).
extern "C" int mi_moe_route(const float* logits, long ld, int T, int E, int top, const float* correction, float scale,
                            float eps, int mode, int renormalize, int groups, int kept_groups, int* chosen, float* weights,
                            float* gate, hipStream_t stream) {
  const RouteArgs a = {logits, ld, T, E, top, correction, scale, eps, mode, renormalize, groups, kept_groups, chosen, weights, gate};
  const int code = check_route(a);
  if (code) return code;
  if (E <= 2 * WAVE) moe_route_kernel<2><<<(T + 3) / 4, 256, 0, stream>>>(a);
  else moe_route_kernel<MOE_PER_LANE><<<(T + 3) / 4, 256, 0, stream>>>(a);
  RETURN_IF_LAUNCH_FAILED();
  return 0;
}

// ---------------------------------------------------------------- rows grouped by expert
struct PlanArgs {
  const int* chosen;
  int entries, top, E, pad, capacity;
  int* source;
  int* place;
  int* tile_expert;
  int* ranks;
  const float* weights;             // with place_weight: the choices' weights, laid beside the places (padding gets 0)
  float* place_weight;
};

// By one workgroup; a choice of E or beyond is an identity expert and gets the place -1.
__device__ __forceinline__ void plan_rows(const PlanArgs& a, int* counts, int* offsets) {
  const int tid = threadIdx.x;
  const int threads = blockDim.x;
  for (int e = tid; e < a.E; e += threads) counts[e] = 0;
  for (int i = tid; i < a.capacity; i += threads) {
    a.source[i] = -1;
    if (a.place_weight) a.place_weight[i] = 0.f;
  }
  for (int t = tid; t < a.capacity / a.pad; t += threads) a.tile_expert[t] = -1;
  __syncthreads();
  for (int i = tid; i < a.entries; i += threads) {
    const int expert = a.chosen[i];
    if (expert < a.E) a.ranks[i] = atomicAdd(&counts[expert], 1);      // (an identity expert's choice stands nowhere)
  }
  __syncthreads();
  // where every expert's places begin: whole tiles, an inclusive sum over the wave in turns of 64 experts
  if (tid < WAVE) {
    int before = 0;
    for (int e0 = 0; e0 < a.E; e0 += WAVE) {
      const int e = e0 + tid;
      const int places = e < a.E ? (counts[e] + a.pad - 1) / a.pad * a.pad : 0;
      int running = places;
#pragma unroll
      for (int offset = 1; offset < WAVE; offset <<= 1) {
        const int other = __shfl_up(running, offset, WAVE);
        if (tid >= offset) running += other;
      }
      if (e < a.E) offsets[e] = before + running - places;
      before += __shfl(running, WAVE - 1, WAVE);
    }
  }
  __syncthreads();
  for (int e = tid; e < a.E; e += threads) {
    const int first = offsets[e] / a.pad;
    const int tiles = (counts[e] + a.pad - 1) / a.pad;
    for (int t = 0; t < tiles; ++t) a.tile_expert[first + t] = e;
  }
  for (int i = tid; i < a.entries; i += threads) {
    const int expert = a.chosen[i];
    if (expert >= a.E) {
      a.place[i] = -1;
      continue;
    }
    const int at = offsets[expert] + a.ranks[i];
    a.source[at] = i / a.top;
    a.place[i] = at;
    if (a.place_weight) a.place_weight[at] = a.weights[i];
  }
}

__global__ void __launch_bounds__(1024) moe_plan_kernel(PlanArgs a) {
  __shared__ int counts[MOE_MAX_EXPERTS];
  __shared__ int offsets[MOE_MAX_EXPERTS];
  plan_rows(a, counts, offsets);
}

static int check_plan(const PlanArgs& a) {
  if (a.place_weight && !a.weights) return ERR_BAD_ARGUMENT;
  if (!a.chosen || !a.source || !a.place || !a.tile_expert || !a.ranks || a.entries <= 0 || a.top <= 0 || a.E <= 0 || a.pad <= 0 ||
      a.capacity % a.pad != 0 || a.capacity < a.entries + a.E * (a.pad - 1))
    return ERR_BAD_ARGUMENT;
  return a.E > MOE_MAX_EXPERTS ? ERR_UNSUPPORTED_SIZE : 0;
}

extern "C" int mi_moe_plan(const int* chosen, int entries, int top, int E, int pad, int capacity, int* source, int* place,
                           int* tile_expert, int* ranks, const float* weights, float* place_weight, hipStream_t stream) {
  const PlanArgs a = {chosen, entries, top, E, pad, capacity, source, place, tile_expert, ranks, weights, place_weight};
  const int code = check_plan(a);
  if (code) return code;
  moe_plan_kernel<<<1, 1024, 0, stream>>>(a);
  RETURN_IF_LAUNCH_FAILED();
  return 0;
}

// Choice and grouping of a step of few tokens in one launch: a wave a token, then the workgroup groups what its waves
// chose (the same workgroup: a barrier makes its own writes visible).
#define ROUTE_PLAN_TOKENS 64
template <int PER_LANE>
__global__ void __launch_bounds__(1024) moe_route_plan_kernel(RouteArgs route, PlanArgs plan) {
  __shared__ int counts[MOE_MAX_EXPERTS];
  __shared__ int offsets[MOE_MAX_EXPERTS];
  for (int token = threadIdx.x / WAVE; token < route.T; token += blockDim.x / WAVE) route_token<PER_LANE>(route, token);
  __threadfence_block();
  __syncthreads();
  plan_rows(plan, counts, offsets);
}

// experts: those with matrices, at most route's E.
extern "C" int mi_moe_route_plan(const float* logits, long ld, int T, int E, int top, const float* correction, float scale,
                                 float eps, int mode, int renormalize, int groups, int kept_groups, int* chosen,
                                 float* weights, float* gate, int experts, int pad, int capacity, int* source, int* place,
                                 int* tile_expert, int* ranks, float* place_weight, hipStream_t stream) {
  const RouteArgs route = {logits, ld, T, E, top, correction, scale, eps, mode, renormalize, groups, kept_groups, chosen, weights, gate};
  const PlanArgs plan = {chosen, T * top, top, experts, pad, capacity, source, place, tile_expert, ranks, weights, place_weight};
  int code = check_route(route);
  if (!code) code = check_plan(plan);
  if (code) return code;
  if (T > ROUTE_PLAN_TOKENS || experts > E) return ERR_UNSUPPORTED_SIZE;
  const int threads = T >= 16 ? 1024 : (T > 4 ? T * WAVE : 4 * WAVE);
  if (E <= 2 * WAVE) moe_route_plan_kernel<2><<<1, threads, 0, stream>>>(route, plan);
  else moe_route_plan_kernel<MOE_PER_LANE><<<1, threads, 0, stream>>>(route, plan);
  RETURN_IF_LAUNCH_FAILED();
  return 0;
}

// ---------------------------------------------------------------- the grouped product
// Tile t of 16 MT places belongs to expert tile_expert[t] (none: the workgroup leaves).  A workgroup owns the
// tile's rows and PAIRS tiles of 16 output features.  GLU: the expert's matrix is [2 I, K], gate rows then up
// rows; out[place, n] = act(gate tile, up tile), n < I.  Places without a row get zeros.  Steps of few rows take
// MT = 1 (every expert's matrix is read once, by as many workgroups as it has tiles of features); prompt portions,
// whose experts get dozens of rows each, MT = 4 and four tiles of features (the rows and the matrix come from the
// caches, 64 x 64 results a workgroup).
template <typename T, typename TO, bool VEC, bool GLU, int MT, int PAIRS>
__global__ void __launch_bounds__(TILE_THREADS)
moe_expert_gemm_kernel(const T* __restrict__ x, long ldx, int x_rows, const T* __restrict__ W, long expert_stride, long ldw,
                       int N, int K, const int* __restrict__ source, const int* __restrict__ tile_expert, int gather,
                       float limit, float alpha, float offset, int squared_relu,
                       const float* __restrict__ row_scale, TO* __restrict__ out, long ldo) {
  __shared__ float red[TILE_WAVES][256];
  const int tile = blockIdx.y;
  const int expert = tile_expert[tile];
  if (expert < 0) return;
  const int tid = threadIdx.x;
  const int r = (tid & (WAVE - 1)) % 16;
  const int width = GLU ? N / 2 : N;
  const long n0 = (long)blockIdx.x * 16 * PAIRS;
  const T* matrix = W + (long)expert * expert_stride;
  constexpr int NT = GLU ? 2 * PAIRS : PAIRS;
  const T* w_row[NT];
  const T* x_row[MT];
#pragma unroll
  for (int p = 0; p < PAIRS; ++p) {
    const long n_row = min(n0 + 16 * p + r, (long)width - 1);
    w_row[p] = matrix + n_row * ldw;
    if (GLU) w_row[NT - PAIRS + p] = matrix + (width + n_row) * ldw;
  }
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    const int place_in = (tile * MT + mt) * 16 + r;
    const long x_at = gather ? max(source[place_in], 0) : place_in;
    x_row[mt] = x + min(x_at, (long)x_rows - 1) * ldx;
  }
  tile_floatx4 acc[NT][MT];
  tile_accumulate<T, MT, NT, VEC>(w_row, x_row, K, acc);
  const int l = tid % 64;
#pragma unroll
  for (int p = 0; p < PAIRS; ++p)
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) {
      const int place = (tile * MT + mt) * 16 + (l % 16);
      const float scale = row_scale ? row_scale[place] : 1.0f;
      float value = tile_reduce(acc[p][mt], red) * scale;
      if (GLU) {
        const float up = tile_reduce(acc[NT - PAIRS + p][mt], red) * scale;
        const float g = fminf(value, limit);
        const float u = fminf(fmaxf(up, -limit), limit);
        value = g / (1.0f + expf(-alpha * g)) * (u + offset);
      } else if (squared_relu) {
        value = fmaxf(value, 0.f);
        value *= value;
      }
      const long n = n0 + 16 * p + 4 * (l / 16) + tid / 64;
      if (n < width) out[(long)place * ldo + n] = from_float<TO>(source[place] >= 0 ? value : 0.f);
    }
}

// Where piece `piece` (0..3) of row `row` of an LDS stage lies: a row is 64 bytes, and the pieces of rows 4 apart
// are swapped among themselves so that the sixteen rows a quarter of a wave reads at once fall into sixteen
// different groups of banks.
__device__ __forceinline__ int stage_slot(int row, int piece) { return row * 4 + (piece ^ ((row >> 2) & 3)); }

// The same product for prompt portions whose rows and matrices are whole 16-byte pieces: a workgroup owns a tile
// of 64 places and 128 rows of its expert's matrix (GLU: 64 gate rows and the 64 up rows that go with them, which
// make 64 outputs; else 128 outputs), walks K one chunk at a time through two LDS stages (the next chunk's pieces
// are asked for before the current one's products), and every wave owns all 64 places and a quarter of the
// features: no sum crosses a wave, a row's result is summed in k order by one lane's accumulator.
template <typename T, typename TO, bool GLU>
__global__ void __launch_bounds__(TILE_THREADS)
moe_expert_gemm_wide_kernel(const T* __restrict__ x, long ldx, int x_rows, const T* __restrict__ W, long expert_stride,
                            long ldw, int N, int K, const int* __restrict__ source, const int* __restrict__ tile_expert,
                            int gather, float limit, float alpha, float offset, int squared_relu,
                            const float* __restrict__ row_scale, TO* __restrict__ out, long ldo) {
  typedef typename TileTraits<T>::Piece Piece;
  constexpr int CHUNK = TileTraits<T>::CHUNK;
  constexpr int PIECE = TileTraits<T>::PIECE;
  constexpr int ROWS = 64, FEATURES = 128;
  __shared__ Piece stage[2][(ROWS + FEATURES) * 4];
  const int tile = blockIdx.y;
  const int expert = tile_expert[tile];
  if (expert < 0) return;
  const int tid = threadIdx.x;
  const int lane = tid & (WAVE - 1);
  const int wave = tid / WAVE;
  const int q = lane / 16;
  const int r = lane % 16;
  const int width = GLU ? N / 2 : N;
  const long n0 = (long)blockIdx.x * (GLU ? 64 : 128);
  const T* matrix = W + (long)expert * expert_stride;
  // what this thread brings into a stage: piece `part` of one row of x and of two rows of the matrix
  const int lrow = tid / 4;
  const int part = tid % 4;
  const int place_in = tile * ROWS + lrow;
  const long x_at = gather ? max(source[place_in], 0) : place_in;
  const T* x_from = x + min(x_at, (long)x_rows - 1) * ldx;
  const T* w_from[2];
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int s = lrow + 64 * j;                                // row of the stage's matrix part
    long feature;
    if (GLU) feature = (j == 0 ? 0 : width) + min(n0 + lrow, (long)width - 1);
    else feature = min(n0 + s, (long)width - 1);
    w_from[j] = matrix + feature * ldw;
  }
  tile_floatx4 acc[2][4];
#pragma unroll
  for (int nt = 0; nt < 2; ++nt)
#pragma unroll
    for (int mt = 0; mt < 4; ++mt) acc[nt][mt] = tile_floatx4{0.f, 0.f, 0.f, 0.f};
  const int chunks = (K + CHUNK - 1) / CHUNK;
  Piece gx = tile_load<T, true>(x_from, PIECE * part, K);
  Piece gw0 = tile_load<T, true>(w_from[0], PIECE * part, K);
  Piece gw1 = tile_load<T, true>(w_from[1], PIECE * part, K);
  stage[0][stage_slot(lrow, part)] = gx;
  stage[0][stage_slot(ROWS + lrow, part)] = gw0;
  stage[0][stage_slot(ROWS + 64 + lrow, part)] = gw1;
  __syncthreads();
  for (int c = 0; c < chunks; ++c) {
    const int cur = c & 1;
    const int k_next = c + 1 < chunks ? (c + 1) * CHUNK + PIECE * part : K;      // past the end: zeros, never used
    gx = tile_load<T, true>(x_from, k_next, K);
    gw0 = tile_load<T, true>(w_from[0], k_next, K);
    gw1 = tile_load<T, true>(w_from[1], k_next, K);
    Piece a[2], b[4];
#pragma unroll
    for (int nt = 0; nt < 2; ++nt) {
      const int row = GLU ? 64 * nt + 16 * wave + r : 32 * wave + 16 * nt + r;
      a[nt] = stage[cur][stage_slot(ROWS + row, q)];
    }
#pragma unroll
    for (int mt = 0; mt < 4; ++mt) b[mt] = stage[cur][stage_slot(16 * mt + r, q)];
#pragma unroll
    for (int nt = 0; nt < 2; ++nt)
#pragma unroll
      for (int mt = 0; mt < 4; ++mt) acc[nt][mt] = tile_mfma(a[nt], b[mt], acc[nt][mt]);
    stage[cur ^ 1][stage_slot(lrow, part)] = gx;
    stage[cur ^ 1][stage_slot(ROWS + lrow, part)] = gw0;
    stage[cur ^ 1][stage_slot(ROWS + 64 + lrow, part)] = gw1;
    __syncthreads();
  }
#pragma unroll
  for (int mt = 0; mt < 4; ++mt) {
    const int place = tile * ROWS + 16 * mt + r;
    const bool live = source[place] >= 0;
    const float scale = row_scale ? row_scale[place] : 1.0f;
    TO* row = out + (long)place * ldo;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if (GLU) {
        const long n = n0 + 16 * wave + 4 * q + i;
        const float g = fminf(acc[0][mt][i] * scale, limit);
        const float u = fminf(fmaxf(acc[1][mt][i] * scale, -limit), limit);
        const float value = g / (1.0f + expf(-alpha * g)) * (u + offset);
        if (n < width) row[n] = from_float<TO>(live ? value : 0.f);
      } else {
#pragma unroll
        for (int nt = 0; nt < 2; ++nt) {
          const long n = n0 + 32 * wave + 16 * nt + 4 * q + i;
          float value = acc[nt][mt][i] * scale;
          if (squared_relu) {
            value = fmaxf(value, 0.f);
            value *= value;
          }
          if (n < width) row[n] = from_float<TO>(live ? value : 0.f);
        }
      }
    }
  }
}

// The widest form, for prompt portions whose experts get hundreds of rows each: 128 places x 128 matrix rows a
// workgroup, every wave a quarter of it as 64 places x 64 matrix rows (GLU: 32 gate rows and their 32 up rows), so
// that eight fragments from LDS feed sixteen matrix instructions.
template <typename T, typename TO, bool GLU>
__global__ void __launch_bounds__(TILE_THREADS)
moe_expert_gemm_widest_kernel(const T* __restrict__ x, long ldx, int x_rows, const T* __restrict__ W, long expert_stride,
                              long ldw, int N, int K, const int* __restrict__ source, const int* __restrict__ tile_expert,
                              int gather, float limit, float alpha, float offset, int squared_relu,
                              const float* __restrict__ row_scale, TO* __restrict__ out, long ldo) {
  typedef typename TileTraits<T>::Piece Piece;
  constexpr int CHUNK = TileTraits<T>::CHUNK;
  constexpr int PIECE = TileTraits<T>::PIECE;
  constexpr int ROWS = 128, FEATURES = 128;
  __shared__ Piece stage[2][(ROWS + FEATURES) * 4];
  const int tile = blockIdx.y;
  const int expert = tile_expert[tile];
  if (expert < 0) return;
  const int tid = threadIdx.x;
  const int lane = tid & (WAVE - 1);
  const int wave = tid / WAVE;
  const int wm = wave / 2;                                     // which 64 places
  const int wn = wave % 2;                                     // which half of the features
  const int q = lane / 16;
  const int r = lane % 16;
  const int width = GLU ? N / 2 : N;
  const long n0 = (long)blockIdx.x * (GLU ? 64 : 128);
  const T* matrix = W + (long)expert * expert_stride;
  const int lrow = tid / 4;
  const int part = tid % 4;
  const T* x_from[2];
  const T* w_from[2];
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int place_in = tile * ROWS + lrow + 64 * j;
    const long x_at = gather ? max(source[place_in], 0) : place_in;
    x_from[j] = x + min(x_at, (long)x_rows - 1) * ldx;
    long feature;
    if (GLU) feature = (j == 0 ? 0 : width) + min(n0 + lrow, (long)width - 1);
    else feature = min(n0 + lrow + 64 * j, (long)width - 1);
    w_from[j] = matrix + feature * ldw;
  }
  tile_floatx4 acc[4][4];
#pragma unroll
  for (int nt = 0; nt < 4; ++nt)
#pragma unroll
    for (int mt = 0; mt < 4; ++mt) acc[nt][mt] = tile_floatx4{0.f, 0.f, 0.f, 0.f};
  const int chunks = (K + CHUNK - 1) / CHUNK;
  Piece gx[2], gw[2];
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    gx[j] = tile_load<T, true>(x_from[j], PIECE * part, K);
    gw[j] = tile_load<T, true>(w_from[j], PIECE * part, K);
    stage[0][stage_slot(lrow + 64 * j, part)] = gx[j];
    stage[0][stage_slot(ROWS + lrow + 64 * j, part)] = gw[j];
  }
  __syncthreads();
  for (int c = 0; c < chunks; ++c) {
    const int cur = c & 1;
    const int k_next = c + 1 < chunks ? (c + 1) * CHUNK + PIECE * part : K;      // past the end: zeros, never used
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      gx[j] = tile_load<T, true>(x_from[j], k_next, K);
      gw[j] = tile_load<T, true>(w_from[j], k_next, K);
    }
    Piece a[4], b[4];
#pragma unroll
    for (int nt = 0; nt < 4; ++nt) {
      // GLU: nt 0, 1 are gate rows, nt 2, 3 the up rows of the same outputs (the stage's second 64 rows)
      const int row = GLU ? 64 * (nt / 2) + 32 * wn + 16 * (nt % 2) + r : 64 * wn + 16 * nt + r;
      a[nt] = stage[cur][stage_slot(ROWS + row, q)];
    }
#pragma unroll
    for (int mt = 0; mt < 4; ++mt) b[mt] = stage[cur][stage_slot(64 * wm + 16 * mt + r, q)];
#pragma unroll
    for (int nt = 0; nt < 4; ++nt)
#pragma unroll
      for (int mt = 0; mt < 4; ++mt) acc[nt][mt] = tile_mfma(a[nt], b[mt], acc[nt][mt]);
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      stage[cur ^ 1][stage_slot(lrow + 64 * j, part)] = gx[j];
      stage[cur ^ 1][stage_slot(ROWS + lrow + 64 * j, part)] = gw[j];
    }
    __syncthreads();
  }
#pragma unroll
  for (int mt = 0; mt < 4; ++mt) {
    const int place = tile * ROWS + 64 * wm + 16 * mt + r;
    const bool live = source[place] >= 0;
    const float scale = row_scale ? row_scale[place] : 1.0f;
    TO* row = out + (long)place * ldo;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if (GLU) {
#pragma unroll
        for (int h = 0; h < 2; ++h) {
          const long n = n0 + 32 * wn + 16 * h + 4 * q + i;
          const float g = fminf(acc[h][mt][i] * scale, limit);
          const float u = fminf(fmaxf(acc[2 + h][mt][i] * scale, -limit), limit);
          const float value = g / (1.0f + expf(-alpha * g)) * (u + offset);
          if (n < width) row[n] = from_float<TO>(live ? value : 0.f);
        }
      } else {
#pragma unroll
        for (int nt = 0; nt < 4; ++nt) {
          const long n = n0 + 64 * wn + 16 * nt + 4 * q + i;
          float value = acc[nt][mt][i] * scale;
          if (squared_relu) {
            value = fmaxf(value, 0.f);
            value *= value;
          }
          if (n < width) row[n] = from_float<TO>(live ? value : 0.f);
        }
      }
    }
  }
}

template <typename T, typename TO>
static void launch_expert_gemm(const T* x, long ldx, int x_rows, const T* W, long expert_stride, long ldw, int N, int K,
                               const int* source, const int* tile_expert, int tiles, int pad, int gather, int activation,
                               float limit, float alpha, float offset, const float* row_scale, TO* out, long ldo,
                               hipStream_t stream) {
  const int glu = activation == 1;
  const int squared_relu = activation == 2;
  constexpr int PIECE = TileTraits<T>::PIECE;
  const bool vec = K % PIECE == 0 && ldx % PIECE == 0 && ldw % PIECE == 0 && expert_stride % PIECE == 0 &&
                   ((unsigned long long)x % 16) == 0 && ((unsigned long long)W % 16) == 0;
  const int width = glu ? N / 2 : N;
#define EXPERT_LAUNCH(VEC_, GLU_, MT_, PAIRS_)                                                                           moe_expert_gemm_kernel<T, TO, VEC_, GLU_, MT_, PAIRS_>                                                                    <<<dim3((unsigned)((width + 16 * PAIRS_ - 1) / (16 * PAIRS_)), (unsigned)tiles), TILE_THREADS, 0, stream>>>(               x, ldx, x_rows, W, expert_stride, ldw, N, K, source, tile_expert, gather, limit, alpha, offset, squared_relu, row_scale, out, ldo)
#define EXPERT_SHAPE(MT_, PAIRS_GLU_, PAIRS_PLAIN_)                                                                      do {                                                                                                                    if (vec && glu) EXPERT_LAUNCH(true, true, MT_, PAIRS_GLU_);                                                            else if (vec) EXPERT_LAUNCH(true, false, MT_, PAIRS_PLAIN_);                                                           else if (glu) EXPERT_LAUNCH(false, true, MT_, PAIRS_GLU_);                                                             else EXPERT_LAUNCH(false, false, MT_, PAIRS_PLAIN_);                                                                 } while (0)
  if (pad == 128) {      // (only plans of rows and matrices in whole pieces are made so wide)
    const dim3 grid((unsigned)((width + (glu ? 64 : 128) - 1) / (glu ? 64 : 128)), (unsigned)tiles);
    if (glu)
      moe_expert_gemm_widest_kernel<T, TO, true><<<grid, TILE_THREADS, 0, stream>>>(
          x, ldx, x_rows, W, expert_stride, ldw, N, K, source, tile_expert, gather, limit, alpha, offset, squared_relu, row_scale, out, ldo);
    else
      moe_expert_gemm_widest_kernel<T, TO, false><<<grid, TILE_THREADS, 0, stream>>>(
          x, ldx, x_rows, W, expert_stride, ldw, N, K, source, tile_expert, gather, limit, alpha, offset, squared_relu, row_scale, out, ldo);
  } else if (pad == 64 && vec) {
    const dim3 grid((unsigned)((width + (glu ? 64 : 128) - 1) / (glu ? 64 : 128)), (unsigned)tiles);
    if (glu)
      moe_expert_gemm_wide_kernel<T, TO, true><<<grid, TILE_THREADS, 0, stream>>>(
          x, ldx, x_rows, W, expert_stride, ldw, N, K, source, tile_expert, gather, limit, alpha, offset, squared_relu, row_scale, out, ldo);
    else
      moe_expert_gemm_wide_kernel<T, TO, false><<<grid, TILE_THREADS, 0, stream>>>(
          x, ldx, x_rows, W, expert_stride, ldw, N, K, source, tile_expert, gather, limit, alpha, offset, squared_relu, row_scale, out, ldo);
  } else if (pad == 64) {
    EXPERT_SHAPE(4, 2, 4);
  } else {
    EXPERT_SHAPE(1, 1, 1);
  }
#undef EXPERT_SHAPE
#undef EXPERT_LAUNCH
}

extern "C" int mi_moe_expert_gemm(const void* x, int dtype, long ldx, int x_rows, const void* W, long expert_stride,
                                  long ldw, int N, int K, const int* source, const int* tile_expert, int tiles, int pad,
                                  int gather, int activation, float limit, float alpha, float offset,
                                  const float* row_scale, void* out, int out_dtype, long ldo, hipStream_t stream) {
  // row_scale (or null): a number for every place that multiplies its row before the product (as the products are linear
  // in the row, the sums before the activation)
  // activation: 0 none, 1 the clamped gated one (the matrix holds gate rows then up rows), 2 max(z, 0)^2
  const int glu = activation == 1;
  if (activation < 0 || activation > 2) return ERR_BAD_ARGUMENT;
  if (!x || !W || !source || !tile_expert || !out || x_rows <= 0 || N <= 0 || K <= 0 || tiles <= 0 || ldx < K || ldw < K ||
      (glu && N % 2) || ldo < (glu ? N / 2 : N))
    return ERR_BAD_ARGUMENT;
  if ((pad != 16 && pad != 64 && pad != 128) || tiles > 65535) return ERR_UNSUPPORTED_SIZE;
  if (pad == 128) {
    const long piece = dtype == DT_F32 ? 4 : 8;
    if (K % piece || ldx % piece || ldw % piece || expert_stride % piece || ((unsigned long long)x % 16) ||
        ((unsigned long long)W % 16))
      return ERR_UNSUPPORTED_SIZE;
  }
  if (dtype == DT_F32 && out_dtype == DT_F32)
    launch_expert_gemm<float, float>((const float*)x, ldx, x_rows, (const float*)W, expert_stride, ldw, N, K, source,
                                     tile_expert, tiles, pad, gather, activation, limit, alpha, offset, row_scale, (float*)out, ldo, stream);
  else if (dtype == DT_BF16 && out_dtype == DT_BF16)
    launch_expert_gemm<bf16_t, bf16_t>((const bf16_t*)x, ldx, x_rows, (const bf16_t*)W, expert_stride, ldw, N, K, source,
                                       tile_expert, tiles, pad, gather, activation, limit, alpha, offset, row_scale, (bf16_t*)out, ldo, stream);
  else if (dtype == DT_BF16 && out_dtype == DT_F32)
    launch_expert_gemm<bf16_t, float>((const bf16_t*)x, ldx, x_rows, (const bf16_t*)W, expert_stride, ldw, N, K, source,
                                      tile_expert, tiles, pad, gather, activation, limit, alpha, offset, row_scale, (float*)out, ldo, stream);
  else
    return ERR_BAD_ARGUMENT;
  RETURN_IF_LAUNCH_FAILED();
  return 0;
}

// ---------------------------------------------------------------- a token's weighted sum
// total[t, i] = sum over the choices k of weights[t, k] * (down[place[t, k], i], or x[t, i] where the place is negative),
// + (gate[t], or one) * shared[t, i]; weights null: every choice counts once.  Without a tail out = total.  With one the sum goes on into the residual stream in
// the same launch: h += tanh(post_alpha total) * post_w + post_b, and (next_w not null) the new rows through the next
// tanh norm, next_out = tanh(next_alpha h) * next_w + next_b.  A thread takes PIECE neighbouring features of a token.
struct CombineTail {
  float* h;
  const float* post_w;
  const float* post_b;
  const float* next_w;
  const float* next_b;
  float post_alpha, next_alpha;
  void* next_out;                   // [T, d] of x's type
};

template <int PIECE>
__device__ __forceinline__ void piece_of(const float* from, float (&to)[PIECE]) {
  if constexpr (PIECE == 1) {
    to[0] = from[0];
  } else {
    const tile_floatx4 piece = *reinterpret_cast<const tile_floatx4*>(from);
#pragma unroll
    for (int j = 0; j < PIECE; ++j) to[j] = piece[j];
  }
}

template <int PIECE>
__device__ __forceinline__ void piece_of(const bf16_t* from, float (&to)[PIECE]) {
  typedef __bf16 four __attribute__((ext_vector_type(4)));
  if constexpr (PIECE == 1) {
    to[0] = (float)from[0];
  } else {
    const four piece = *reinterpret_cast<const four*>(from);
#pragma unroll
    for (int j = 0; j < PIECE; ++j) to[j] = (float)piece[j];
  }
}

template <typename TS, typename TX, int PIECE>
__global__ void __launch_bounds__(256)
moe_combine_kernel(const float* __restrict__ down, long ld, const int* __restrict__ place, const float* __restrict__ weights,
                   int top, const TX* __restrict__ x, long x_ld, const TS* __restrict__ shared, long shared_ld,
                   const float* __restrict__ gate, float* __restrict__ out, int d, long total_pieces, CombineTail tail) {
  const long index = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (index >= total_pieces) return;
  const int pieces = d / PIECE;
  const long token = index / pieces;
  const int i = (int)(index - token * pieces) * PIECE;
  float own[PIECE], extra[PIECE], total[PIECE], stream[PIECE], pw[PIECE], pb[PIECE], nw[PIECE], nb[PIECE];
#pragma unroll
  for (int j = 0; j < PIECE; ++j) own[j] = extra[j] = total[j] = 0.f;
  if (x) piece_of<PIECE>(x + token * x_ld + i, own);
  if (shared) piece_of<PIECE>(shared + token * shared_ld + i, extra);
  if (tail.h) {
    piece_of<PIECE>(tail.h + token * d + i, stream);
    piece_of<PIECE>(tail.post_w + i, pw);
    piece_of<PIECE>(tail.post_b + i, pb);
    if (tail.next_w) {
      piece_of<PIECE>(tail.next_w + i, nw);
      piece_of<PIECE>(tail.next_b + i, nb);
    }
  }
  for (int k0 = 0; k0 < top; k0 += 4) {
    // four choices' rows asked for at once; a choice past the last reads the last again and weighs nothing
    float value[4][PIECE], weight[4];
    int at[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int k = min(k0 + u, top - 1);
      at[u] = place[token * top + k];
      weight[u] = k0 + u < top ? (weights ? weights[token * top + k] : 1.0f) : 0.f;
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) piece_of<PIECE>(down + (long)max(at[u], 0) * ld + i, value[u]);
#pragma unroll
    for (int u = 0; u < 4; ++u)
      if (k0 + u < top) {
#pragma unroll
        for (int j = 0; j < PIECE; ++j) total[j] = fmaf(weight[u], at[u] < 0 ? own[j] : value[u][j], total[j]);
      }
  }
  if (shared) {
    const float share = gate ? gate[token] : 1.0f;
#pragma unroll
    for (int j = 0; j < PIECE; ++j) total[j] = fmaf(share, extra[j], total[j]);
  }
  if (!tail.h) {
    if constexpr (PIECE == 1) out[token * d + i] = total[0];
    else *reinterpret_cast<tile_floatx4*>(out + token * d + i) = tile_floatx4{total[0], total[1], total[2], total[3]};
    return;
  }
#pragma unroll
  for (int j = 0; j < PIECE; ++j) stream[j] += tanh_norm_f(total[j], tail.post_alpha, pw[j], pb[j]);
  if constexpr (PIECE == 1) tail.h[token * d + i] = stream[0];
  else *reinterpret_cast<tile_floatx4*>(tail.h + token * d + i) = tile_floatx4{stream[0], stream[1], stream[2], stream[3]};
  if (!tail.next_w) return;
  TX* next = (TX*)tail.next_out + token * d + i;
  if constexpr (PIECE == 1) {
    next[0] = from_float<TX>(tanh_norm_f(stream[0], tail.next_alpha, nw[0], nb[0]));
  } else {
    typedef TX four __attribute__((ext_vector_type(4)));
    four piece;
#pragma unroll
    for (int j = 0; j < 4; ++j) piece[j] = from_float<TX>(tanh_norm_f(stream[j], tail.next_alpha, nw[j], nb[j]));
    *reinterpret_cast<four*>(next) = piece;
  }
}

// out, or (h not null) the tail, whose next rows have x_dtype.
extern "C" int mi_moe_combine(const float* down, long ld, const int* place, const float* weights, int top, const void* x,
                              int x_dtype, long x_ld, const void* shared, int shared_dtype, long shared_ld,
                              const float* gate, float* out, int T, int d, float* h, const float* post_w,
                              const float* post_b, float post_alpha, const float* next_w, const float* next_b,
                              float next_alpha, void* next_out, hipStream_t stream) {
  if (!down || !place || T <= 0 || d <= 0 || top <= 0 || ld < d || (shared && shared_ld < d) || (x && x_ld < d))
    return ERR_BAD_ARGUMENT;
  if (h ? (!post_w || !post_b || (next_w && (!next_b || !next_out))) : !out) return ERR_BAD_ARGUMENT;
  const CombineTail tail = {h, post_w, post_b, next_w, next_b, post_alpha, next_alpha, next_out};
  const uintptr_t addresses = (uintptr_t)down | (uintptr_t)x | (uintptr_t)shared | (uintptr_t)out | (uintptr_t)h | (uintptr_t)post_w |
                              (uintptr_t)post_b | (uintptr_t)next_w | (uintptr_t)next_b | (uintptr_t)next_out;
  const bool fours = d % 4 == 0 && ld % 4 == 0 && x_ld % 4 == 0 && shared_ld % 4 == 0 && addresses % 16 == 0;
  const long pieces = (long)T * d / (fours ? 4 : 1);
  const int block = pieces <= 64 * 1024 ? WAVE : 256;
  const long blocks = (pieces + block - 1) / block;
  if (blocks > 0x7fffffffL) return ERR_UNSUPPORTED_SIZE;
#define COMBINE_PIECE(TS_, TX_, PIECE_)                                                                                \
  moe_combine_kernel<TS_, TX_, PIECE_><<<(unsigned)blocks, block, 0, stream>>>(                                        \
      down, ld, place, weights, top, (const TX_*)x, x_ld, (const TS_*)shared, shared_ld, gate, out, d, pieces, tail)
#define COMBINE_LAUNCH(TS_, TX_)                                                                                       \
  do {                                                                                                                 \
    if (fours) COMBINE_PIECE(TS_, TX_, 4);                                                                             \
    else COMBINE_PIECE(TS_, TX_, 1);                                                                                   \
  } while (0)
  if (shared_dtype == DT_F32 && x_dtype == DT_F32) COMBINE_LAUNCH(float, float);
  else if (shared_dtype == DT_F32 && x_dtype == DT_BF16) COMBINE_LAUNCH(float, bf16_t);
  else if (shared_dtype == DT_BF16 && x_dtype == DT_F32) COMBINE_LAUNCH(bf16_t, float);
  else if (shared_dtype == DT_BF16 && x_dtype == DT_BF16) COMBINE_LAUNCH(bf16_t, bf16_t);
  else return ERR_BAD_ARGUMENT;
#undef COMBINE_LAUNCH
#undef COMBINE_PIECE
  RETURN_IF_LAUNCH_FAILED();
  return 0;
}
