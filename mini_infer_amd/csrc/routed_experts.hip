// A feed-forward of routed experts: every token goes through `top` of the experts, chosen by a
// router, and the results are added with the router's weights.
//
//   route_top_k         per token: logits z = R x (R float32, sums float32; 64-bit in the 32-bit
//                       engine), scores s = softmax(z) over all router outputs or logistic(z) one by
//                       one, choice = s + correction, the `top` largest choices (the lower index wins
//                       a tie; logistic scores without a correction are ranked by z itself, of which
//                       they are a rising function); leaves the chosen indices and their weights
//                       s * route_scale (not renormalized), and, where a gate row is given,
//                       logistic(gate . x) for a shared expert.  With scores of the third kind the
//                       correction is a bias of the logits, the largest biased logits are chosen and
//                       weights are route_scale times the softmax over the chosen ones alone.
//   route_logits, route_list   the same and the list of pairs by expert, for few bfloat16 tokens.
//   expert_gate_up      few rows: for every (token, chosen expert) pair the expert's first product and
//                       its activation, the weights read by expert index.
//   expert_down_combine few rows: y[t] = sum_k w[t, k] * (W_down[e_k] act[t, k])  (+ shared_gate[t] *
//                       shared[t]); a chosen index past the real experts is an identity expert,
//                       whose output is the token's input row itself.
//   expert_combine      many rows: the same sum over rows of expert outputs that were made expert
//                       by expert (sorted by expert; `where` maps a pair to its sorted row).
//                       (A shared expert's rows without a shared_gate are added as they are.)
//
// Expert weights are stacked: gate|up [experts, 2 * ff, width] (an expert's gate rows, then its up
// rows), or up [experts, ff, width] where experts have no gate; down [experts, width, ff].
//
// What the first product of an expert ends with (MODE):
//   EXPERT_SILU_GATED    silu(gate . x) * (up . x)
//   EXPERT_SQUARED_RELU  relu(w * (up . x))^2, w the pair's router weight: the weight multiplies what the
//                        expert reads, and W (w x) = w (W x), so no weighted copy of the rows is made
// and EXPERT_PLAIN, the second product alone.
#include "common.h"

#include <math.h>

namespace {

template <typename T>
struct SumOf {
  using type = float;
};
template <>
struct SumOf<float> {
  using type = double;
};

__device__ __forceinline__ float lanes_total(float v) { return wave_sum(v); }
__device__ __forceinline__ double lanes_total(double v) {
#pragma unroll
  for (int off = MI_WAVE / 2; off > 0; off >>= 1) v += __shfl_xor(v, off, MI_WAVE);
  return v;
}

__device__ __forceinline__ float exp_of(float z) { return expf(z); }
__device__ __forceinline__ double exp_of(double z) { return exp(z); }

#define MI_ROUTER_MAX_OUTPUTS 1024

enum ExpertMode { EXPERT_PLAIN = 0, EXPERT_SILU_GATED = 1, EXPERT_SQUARED_RELU = 2 };

// what is written for a feature whose sums are `a` (and, gated, `b`), float32 or 64-bit; `weight` is the pair's
template <typename T, int MODE, typename A>
__device__ __forceinline__ T expert_feature(A a, A b, A weight) {
  if constexpr (MODE == EXPERT_SILU_GATED) {
    // the two products as the element type holds them, then silu(gate) * up
    const A g = (A)to_f32(from_f32<T>((float)a)), u = (A)to_f32(from_f32<T>((float)b));
    return from_f32<T>((float)(g / ((A)1 + exp_of(-g)) * u));
  } else if constexpr (MODE == EXPERT_SQUARED_RELU) {
    const A z = weight * a;
    return from_f32<T>((float)(z > (A)0 ? z * z : (A)0));
  } else {
    return from_f32<T>((float)a);
  }
}

// How a token's scores are made of its logits.
enum RouterScores { SCORES_SOFTMAX = 0, SCORES_LOGISTIC = 1, SCORES_CHOSEN_SOFTMAX = 2 };

// A wave ranks a token's outputs, lane l those with e % 64 == l: the `top` largest choices and their weights.
// `mine`: the token's logits in LDS, this wave's own (spent here: chosen ones are marked).
template <typename A>
__device__ __forceinline__ void rank_outputs(A* mine, const float* __restrict__ correction, int* __restrict__ chosen,
                                             float* __restrict__ weights, int outputs, int top, float route_scale,
                                             int scores, int lane) {
  const A taken = -(A)INFINITY;
  A most = taken, total_exp = 0;
  const bool logistic = scores == SCORES_LOGISTIC;
  if (scores == SCORES_CHOSEN_SOFTMAX) {
    // biased logits are what is ranked and what the weights are made of; the sum of exponentials is known
    // only when all are chosen, so the weights are divided by it at the end
    if (correction != nullptr) {
      for (int e = lane; e < outputs; e += MI_WAVE) mine[e] += (A)correction[e];
    }
    correction = nullptr;
  } else if (!logistic) {
    for (int e = lane; e < outputs; e += MI_WAVE) most = mine[e] > most ? mine[e] : most;
#pragma unroll
    for (int off = MI_WAVE / 2; off > 0; off >>= 1) {
      const A other = __shfl_xor(most, off, MI_WAVE);
      most = other > most ? other : most;
    }
    for (int e = lane; e < outputs; e += MI_WAVE) total_exp += exp_of(mine[e] - most);
    total_exp = lanes_total(total_exp);
  }
  const A inv = (A)1 / total_exp;  // (softmax)
  A first_choice = taken;
  auto score_of = [&](A logit) { return logistic ? (A)1 / ((A)1 + exp_of(-logit)) : exp_of(logit - most) * inv; };
  // the choice is made on score + correction (without one on the logit, of which every score is a rising
  // function), the weight is the score alone
  for (int k = 0; k < top; ++k) {
    int best = outputs;
    A best_choice = taken;
    for (int e = lane; e < outputs; e += MI_WAVE) {
      const A logit = mine[e];
      if (logit == taken) continue;
      const A choice = correction != nullptr ? score_of(logit) + (A)correction[e] : logit;
      if (best == outputs || choice > best_choice) best = e, best_choice = choice;
    }
#pragma unroll
    for (int off = MI_WAVE / 2; off > 0; off >>= 1) {
      const A other = __shfl_xor(best_choice, off, MI_WAVE);
      const int index = __shfl_xor(best, off, MI_WAVE);
      if (index < outputs && (best == outputs || other > best_choice || (other == best_choice && index < best))) best = index, best_choice = other;
    }
    if (best == outputs) best = 0;  // (more infinite logits than there are choices)
    if (scores == SCORES_CHOSEN_SOFTMAX) {
      if (k == 0) first_choice = best_choice;  // (the largest: no exponential below passes 1)
      const A share = exp_of(best_choice - first_choice);
      total_exp += share;
      if (lane == 0) {
        chosen[k] = best;
        weights[k] = (float)share;
      }
    } else if (lane == 0) {
      chosen[k] = best;
      weights[k] = (float)(score_of(mine[best]) * (A)route_scale);
    }
    // (the same lane that ranks this output marks it; within a wave LDS is read and written in program order)
    __builtin_amdgcn_wave_barrier();
    if (lane == best % MI_WAVE) mine[best] = taken;
    __builtin_amdgcn_wave_barrier();
  }
  if (scores == SCORES_CHOSEN_SOFTMAX && lane == 0) {
    for (int k = 0; k < top; ++k) weights[k] = (float)((A)weights[k] / total_exp * (A)route_scale);
  }
}

// R tokens a block: their rows wait in LDS while every wave walks router rows (16 bytes a lane, each
// router row read once for all R tokens), then wave r ranks token r's outputs.
template <typename T, int R>
__global__ __launch_bounds__(1024) void route_top_k_kernel(
    const T* __restrict__ x, int64_t x_stride, const float* __restrict__ router, const float* __restrict__ correction,
    const float* __restrict__ gate_row, int* __restrict__ chosen, float* __restrict__ weights,
    float* __restrict__ shared_gate, int num_tokens, int width, int outputs, int top, float route_scale, int scores) {
  using A = typename SumOf<T>::type;
  extern __shared__ __align__(16) unsigned char lds_bytes[];
  A* z = reinterpret_cast<A*>(lds_bytes);                         // [R][outputs + 1]
  T* rows = reinterpret_cast<T*>(z + (size_t)R * (outputs + 1));  // [R][width]
  const int t0 = blockIdx.x * R;
  constexpr int V = 16 / sizeof(T);
  const size_t rows_at = (size_t)R * (outputs + 1) * sizeof(A);
  if (width % V == 0 && x_stride % V == 0 && ((uintptr_t)x % 16) == 0 && rows_at % 16 == 0) {  // 16 bytes a thread
    for (int i = threadIdx.x * V; i < R * width; i += blockDim.x * V) {
      const int r = i / width, c = i % width;
      uint4 got = make_uint4(0, 0, 0, 0);
      if (t0 + r < num_tokens) got = *reinterpret_cast<const uint4*>(x + (int64_t)(t0 + r) * x_stride + c);
      *reinterpret_cast<uint4*>(rows + i) = got;
    }
  } else {
    for (int i = threadIdx.x; i < R * width; i += blockDim.x) {
      const int r = i / width, c = i % width;
      rows[i] = (t0 + r < num_tokens) ? x[(int64_t)(t0 + r) * x_stride + c] : from_f32<T>(0.f);
    }
  }
  __syncthreads();
  const int wave = threadIdx.x / MI_WAVE, lane = threadIdx.x % MI_WAVE, waves = blockDim.x / MI_WAVE;
  const int total = outputs + (gate_row != nullptr ? 1 : 0);
  const bool vec = width % 4 == 0 && ((uintptr_t)router % 16) == 0 && (gate_row == nullptr || ((uintptr_t)gate_row % 16) == 0);
  for (int e = wave; e < total; e += waves) {
    const float* w = e < outputs ? router + (int64_t)e * width : gate_row;
    A sum[R];
#pragma unroll
    for (int r = 0; r < R; ++r) sum[r] = 0;
    if (vec) {
      // (BATCH pieces of the router row are asked for before the first is used)
      constexpr int BATCH = 8;
      for (int c0 = lane * 4; c0 < width; c0 += MI_WAVE * 4 * BATCH) {
        float4 w4[BATCH];
#pragma unroll
        for (int i = 0; i < BATCH; ++i) {
          const int c = c0 + i * MI_WAVE * 4;
          w4[i] = c < width ? *reinterpret_cast<const float4*>(w + c) : make_float4(0.f, 0.f, 0.f, 0.f);
        }
#pragma unroll
        for (int i = 0; i < BATCH; ++i) {
          const int c = c0 + i * MI_WAVE * 4;
          if (c >= width) continue;
#pragma unroll
          for (int r = 0; r < R; ++r) {
            float xv[4];
            mi_load_cols<T, 4>(rows + (size_t)r * width + c, xv);
            sum[r] += (A)w4[i].x * (A)xv[0] + (A)w4[i].y * (A)xv[1] + (A)w4[i].z * (A)xv[2] + (A)w4[i].w * (A)xv[3];
          }
        }
      }
    } else {
      for (int c = lane; c < width; c += MI_WAVE) {
        const A wc = (A)w[c];
#pragma unroll
        for (int r = 0; r < R; ++r) sum[r] += wc * (A)to_f32(rows[(size_t)r * width + c]);
      }
    }
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const A all = lanes_total(sum[r]);
      if (lane == 0) z[r * (outputs + 1) + e] = all;
    }
  }
  __syncthreads();
  for (int r = wave; r < R; r += waves) {
    const int t = t0 + r;
    if (t >= num_tokens) break;
    A* mine = z + r * (outputs + 1);
    if (gate_row != nullptr && lane == 0) shared_gate[t] = (float)((A)1 / ((A)1 + exp_of(-mine[outputs])));
    rank_outputs<A>(mine, correction, chosen + (int64_t)t * top, weights + (int64_t)t * top, outputs, top, route_scale, scores, lane);
  }
}

// a wave's dot product of a weight row with a vector kept in LDS in the element type
template <typename T, typename A>
__device__ __forceinline__ A dot_lds(const T* __restrict__ w, const T* __restrict__ v, int n, int lane) {
  A sum = 0;
  if (n % 8 == 0 && ((uintptr_t)w % 16) == 0) {
    constexpr int V = 16 / sizeof(T);
    for (int c = lane * V; c < n; c += MI_WAVE * V) {
      alignas(16) T a[V];
      *reinterpret_cast<uint4*>(a) = *reinterpret_cast<const uint4*>(w + c);
#pragma unroll
      for (int j = 0; j < V; ++j) sum += (A)to_f32(a[j]) * (A)to_f32(v[c + j]);
    }
  } else {
    for (int c = lane; c < n; c += MI_WAVE) sum += (A)to_f32(w[c]) * (A)to_f32(v[c]);
  }
  return lanes_total(sum);
}

#define MI_EXPERT_FEATURES 16  // features (or columns) a block of four waves makes

template <typename T, int MODE>
__global__ __launch_bounds__(256) void expert_gate_up_kernel(
    const T* __restrict__ x, int64_t x_stride, const T* __restrict__ gate_up, const int* __restrict__ chosen,
    const float* __restrict__ pair_weight, T* __restrict__ act, int width, int ff, int experts, int top) {
  using A = typename SumOf<T>::type;
  extern __shared__ __align__(16) unsigned char lds_bytes[];
  T* row = reinterpret_cast<T*>(lds_bytes);
  const int pair = blockIdx.x;
  const int e = chosen[pair];
  if (e < 0 || e >= experts) return;  // an identity expert: nothing to make (the whole block leaves)
  const T* src = x + (int64_t)(pair / top) * x_stride;
  for (int c = threadIdx.x; c < width; c += blockDim.x) row[c] = src[c];
  __syncthreads();
  const int wave = threadIdx.x / MI_WAVE, lane = threadIdx.x % MI_WAVE, waves = blockDim.x / MI_WAVE;
  constexpr bool GATED = MODE == EXPERT_SILU_GATED;
  const T* w = gate_up + (int64_t)e * (GATED ? 2 : 1) * ff * width;
  const A weight = MODE == EXPERT_SQUARED_RELU && pair_weight != nullptr ? (A)pair_weight[pair] : (A)1;
  const int first = blockIdx.y * MI_EXPERT_FEATURES;
  for (int f = first + wave; f < min(first + MI_EXPERT_FEATURES, ff); f += waves) {
    const A g = dot_lds<T, A>(w + (int64_t)f * width, row, width, lane);
    const A u = GATED ? dot_lds<T, A>(w + (int64_t)(ff + f) * width, row, width, lane) : (A)0;
    if (lane == 0) act[(int64_t)pair * ff + f] = expert_feature<T, MODE, A>(g, u, weight);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void expert_down_combine_kernel(
    const T* __restrict__ act, const T* __restrict__ down, const int* __restrict__ chosen, const float* __restrict__ weights,
    const T* __restrict__ x, int64_t x_stride, const T* __restrict__ shared, int64_t shared_stride,
    const float* __restrict__ shared_gate, T* __restrict__ out, int width, int ff, int experts, int top) {
  using A = typename SumOf<T>::type;
  extern __shared__ __align__(16) unsigned char lds_bytes[];
  T* rows = reinterpret_cast<T*>(lds_bytes);  // [top][ff]
  const int t = blockIdx.x;
  for (int i = threadIdx.x; i < top * ff; i += blockDim.x) {
    const int e = chosen[(int64_t)t * top + i / ff];
    rows[i] = (e >= 0 && e < experts) ? act[(int64_t)t * top * ff + i] : from_f32<T>(0.f);
  }
  __syncthreads();
  const int wave = threadIdx.x / MI_WAVE, lane = threadIdx.x % MI_WAVE, waves = blockDim.x / MI_WAVE;
  const int first = blockIdx.y * MI_EXPERT_FEATURES;
  for (int c = first + wave; c < min(first + MI_EXPERT_FEATURES, width); c += waves) {
    A sum = 0;
    for (int k = 0; k < top; ++k) {
      const int e = chosen[(int64_t)t * top + k];
      const A weight = weights != nullptr ? (A)weights[(int64_t)t * top + k] : (A)1;
      if (e >= experts) {
        sum += weight * (A)to_f32(x[(int64_t)t * x_stride + c]);
      } else if (e >= 0) {
        const A y = dot_lds<T, A>(down + ((int64_t)e * width + c) * ff, rows + (int64_t)k * ff, ff, lane);
        sum += weight * (A)to_f32(from_f32<T>((float)y));
      }
    }
    if (shared != nullptr) sum += (shared_gate != nullptr ? (A)shared_gate[t] : (A)1) * (A)to_f32(shared[(int64_t)t * shared_stride + c]);
    if (lane == 0) out[(int64_t)t * width + c] = from_f32<T>((float)sum);
  }
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void expert_combine_kernel(
    const T* __restrict__ made, const int* __restrict__ where, const int* __restrict__ chosen,
    const float* __restrict__ weights, const T* __restrict__ x, int64_t x_stride, const T* __restrict__ shared,
    int64_t shared_stride, const float* __restrict__ shared_gate, T* __restrict__ out, int width, int experts, int top) {
  using A = typename SumOf<T>::type;
  const int t = blockIdx.x;
  for (int c = threadIdx.x * VEC; c < width; c += blockDim.x * VEC) {
    A sum[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) sum[j] = 0;
    for (int k = 0; k < top; ++k) {
      const int64_t pair = (int64_t)t * top + k;
      const int e = chosen[pair];
      if (e < 0) continue;
      const T* src = e >= experts ? x + (int64_t)t * x_stride : made + (int64_t)(where != nullptr ? where[pair] : pair) * width;
      float v[VEC];
      mi_load_cols<T, VEC>(src + c, v);
      const A weight = weights != nullptr ? (A)weights[pair] : (A)1;
#pragma unroll
      for (int j = 0; j < VEC; ++j) sum[j] += weight * (A)v[j];
    }
    float r[VEC];
    if (shared != nullptr) {
      mi_load_cols<T, VEC>(shared + (int64_t)t * shared_stride + c, r);
      const A g = shared_gate != nullptr ? (A)shared_gate[t] : (A)1;
#pragma unroll
      for (int j = 0; j < VEC; ++j) sum[j] += g * (A)r[j];
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) r[j] = (float)sum[j];
    mi_store_cols<T, VEC>(out + (int64_t)t * width + c, r);
  }
}

inline bool is_aligned16(const void* p) { return ((uintptr_t)p % 16) == 0; }

// ---------------------------------------------------------------------------------------------
// Expert by expert, for steps of few rows that the host knows nothing about (recorded steps):
//   expert_sort      one block: the (token, choice) pairs counted per chosen expert and listed expert
//                    by expert (`listed` [pairs], `first` [experts + 1]; identity experts are left out).
//   expert_rows      a block owns one expert and a tile of FT of its output features, and walks the
//                    expert's listed pairs R rows at a time: the rows wait in LDS, every wave streams
//                    its features' weight rows once for all R rows (16 bytes a lane) and keeps
//                    R sums a weight row.  GATED: features come in pairs (gate row f, up row
//                    ff + f) and silu(gate) * up is what is written; else the plain product.
// So an expert's weights are read once per R of its rows, whatever the number of pairs.
// ---------------------------------------------------------------------------------------------

#define MI_SORT_MAX_EXPERTS 1024

// The pairs counted (`count` [experts + 1] in LDS, one an expert) become the experts' places: `first` and, in
// `count`, where an expert's next pair goes.  The block's first wave, 64 experts a turn.
__device__ __forceinline__ void place_experts(int* count, int* __restrict__ first, int experts) {
  if (threadIdx.x >= MI_WAVE) return;
  const int lane = threadIdx.x;
  int at = 0;
  for (int base = 0; base < experts; base += MI_WAVE) {
    const int n = base + lane < experts ? count[base + lane] : 0;
    int upto = n;
#pragma unroll
    for (int off = 1; off < MI_WAVE; off <<= 1) {
      const int other = __shfl_up(upto, off, MI_WAVE);
      if (lane >= off) upto += other;
    }
    if (base + lane < experts) {
      first[base + lane] = at + upto - n;
      count[base + lane] = at + upto - n;
    }
    at += __shfl(upto, MI_WAVE - 1, MI_WAVE);
  }
  if (lane == 0) first[experts] = at;
}

__global__ __launch_bounds__(1024) void expert_sort_kernel(const int* __restrict__ chosen, int* __restrict__ listed,
                                                           int* __restrict__ first, int pairs, int experts) {
  __shared__ int count[MI_SORT_MAX_EXPERTS + 1];
  for (int e = threadIdx.x; e <= experts; e += blockDim.x) count[e] = 0;
  __syncthreads();
  for (int p = threadIdx.x; p < pairs; p += blockDim.x) {
    const int e = chosen[p];
    if (e >= 0 && e < experts) atomicAdd(&count[e], 1);
  }
  __syncthreads();
  place_experts(count, first, experts);
  __syncthreads();
  // (pairs of one expert in any order: each pair's result is its own)
  for (int p = threadIdx.x; p < pairs; p += blockDim.x) {
    const int e = chosen[p];
    if (e >= 0 && e < experts) listed[atomicAdd(&count[e], 1)] = p;
  }
}

// The router for few tokens (bfloat16), where one block a handful of tokens would leave the router's matrix to
// the bandwidth of a CU or two: `route_logits` makes one output for eight tokens a block, its four waves sharing
// the row, and `route_list` ranks all tokens, a wave a token, and lists the pairs by expert in the same launch.
#define MI_ROUTE_FEW_TOKENS 32
#define MI_ROUTE_FEW_PAIRS 2048

__global__ __launch_bounds__(256) void route_logits_kernel(const bf16_t* __restrict__ x, int64_t x_stride,
                                                           const float* __restrict__ router,
                                                           const float* __restrict__ gate_row, float* __restrict__ logits,
                                                           int num_tokens, int width, int outputs, int total) {
  constexpr int TOKENS = 8;
  __shared__ float meet[3][TOKENS];
  const int e = blockIdx.x, t0 = blockIdx.y * TOKENS;
  const int wave = threadIdx.x / MI_WAVE, lane = threadIdx.x % MI_WAVE;
  const float* w = e < outputs ? router + (int64_t)e * width : gate_row;
  float sum[TOKENS];
#pragma unroll
  for (int t = 0; t < TOKENS; ++t) sum[t] = 0.f;
  constexpr int BATCH = 2;
  for (int c0 = threadIdx.x * 4; c0 < width; c0 += 1024 * BATCH) {
    float wv[BATCH][4], xv[BATCH][TOKENS][4];
#pragma unroll
    for (int i = 0; i < BATCH; ++i) {
      const int c = min(c0 + i * 1024, width - 4);  // (past the row: its last columns again, weighed with zero)
      mi_load_cols<float, 4>(w + c, wv[i]);
      if (c0 + i * 1024 >= width) wv[i][0] = wv[i][1] = wv[i][2] = wv[i][3] = 0.f;
#pragma unroll
      for (int t = 0; t < TOKENS; ++t) mi_load_cols<bf16_t, 4>(x + (int64_t)min(t0 + t, num_tokens - 1) * x_stride + c, xv[i][t]);
    }
#pragma unroll
    for (int i = 0; i < BATCH; ++i)
#pragma unroll
      for (int t = 0; t < TOKENS; ++t)
        sum[t] += wv[i][0] * xv[i][t][0] + wv[i][1] * xv[i][t][1] + wv[i][2] * xv[i][t][2] + wv[i][3] * xv[i][t][3];
  }
#pragma unroll
  for (int t = 0; t < TOKENS; ++t) sum[t] = wave_sum(sum[t]);
  if (wave > 0 && lane == 0) {
#pragma unroll
    for (int t = 0; t < TOKENS; ++t) meet[wave - 1][t] = sum[t];
  }
  __syncthreads();
  if (wave == 0 && lane == 0) {
#pragma unroll
    for (int t = 0; t < TOKENS; ++t)
      if (t0 + t < num_tokens) logits[(int64_t)(t0 + t) * total + e] = sum[t] + meet[0][t] + meet[1][t] + meet[2][t];
  }
}

__global__ __launch_bounds__(1024) void route_list_kernel(const float* __restrict__ logits, const float* __restrict__ correction,
                                                          int* __restrict__ chosen, float* __restrict__ weights,
                                                          float* __restrict__ shared_gate, int* __restrict__ listed,
                                                          int* __restrict__ first, int num_tokens, int outputs, int total,
                                                          int experts, int top, float route_scale, int scores) {
  extern __shared__ __align__(16) unsigned char lds_bytes[];
  float* z = reinterpret_cast<float*>(lds_bytes);                        // [waves][outputs]
  __shared__ int count[MI_SORT_MAX_EXPERTS + 1];
  const int wave = threadIdx.x / MI_WAVE, lane = threadIdx.x % MI_WAVE, waves = blockDim.x / MI_WAVE;
  for (int e = threadIdx.x; e <= experts; e += blockDim.x) count[e] = 0;
  for (int t = wave; t < num_tokens; t += waves) {
    float* mine = z + wave * outputs;
    for (int e = lane; e < outputs; e += MI_WAVE) mine[e] = logits[(int64_t)t * total + e];
    __builtin_amdgcn_wave_barrier();
    if (total > outputs && lane == 0) shared_gate[t] = 1.f / (1.f + expf(-logits[(int64_t)t * total + outputs]));
    rank_outputs<float>(mine, correction, chosen + t * top, weights + t * top, outputs, top, route_scale, scores, lane);
  }
  __syncthreads();  // (what this block's waves have written to `chosen` is there for all of them)
  const int pairs = num_tokens * top;
  for (int p = threadIdx.x; p < pairs; p += blockDim.x) {
    const int e = chosen[p];
    if (e >= 0 && e < experts) atomicAdd(&count[e], 1);
  }
  __syncthreads();
  place_experts(count, first, experts);
  __syncthreads();
  for (int p = threadIdx.x; p < pairs; p += blockDim.x) {
    const int e = chosen[p];
    if (e >= 0 && e < experts) listed[atomicAdd(&count[e], 1)] = p;
  }
}

template <typename T, int R, int MODE>
__global__ __launch_bounds__(256) void expert_rows_kernel(
    const T* __restrict__ src, int64_t src_stride, int src_div, const T* __restrict__ weight, int64_t expert_stride,
    const int* __restrict__ listed, const int* __restrict__ first, const float* __restrict__ pair_weight,
    T* __restrict__ out, int64_t out_stride, int k_dim, int features) {
  using A = typename SumOf<T>::type;
  constexpr bool GATED = MODE == EXPERT_SILU_GATED;
  constexpr int FW = 4;             // features a wave
  constexpr int WR = GATED ? 2 : 1;  // weight rows a feature
  constexpr int V = 16 / sizeof(T);
  extern __shared__ __align__(16) unsigned char lds_bytes[];
  T* rows = reinterpret_cast<T*>(lds_bytes);  // [R][k_dim]
  const int e = blockIdx.y;  // (feature tiles run fastest: a chosen expert's blocks follow one another and spread over all XCDs)
  const int begin = first[e], end = first[e + 1];
  if (begin >= end) return;  // nobody chose this expert (the whole block leaves)
  const int wave = threadIdx.x / MI_WAVE, lane = threadIdx.x % MI_WAVE;
  const int f0 = (blockIdx.x * (blockDim.x / MI_WAVE) + wave) * FW;
  const T* w = weight + (int64_t)e * expert_stride;
  for (int chunk = begin; chunk < end; chunk += R) {
    const int n = min(R, end - chunk);
    __syncthreads();
    for (int i = threadIdx.x * V; i < R * k_dim; i += blockDim.x * V) {
      const int r = i / k_dim, c = i % k_dim;  // (V divides k_dim)
      uint4 got = make_uint4(0, 0, 0, 0);
      if (r < n) got = *reinterpret_cast<const uint4*>(src + (int64_t)(listed[chunk + r] / src_div) * src_stride + c);
      *reinterpret_cast<uint4*>(rows + i) = got;
    }
    __syncthreads();
    if (f0 >= features) continue;  // (a wave past the last feature still helps to stage rows)
    A sum[FW][WR][R];
#pragma unroll
    for (int f = 0; f < FW; ++f)
#pragma unroll
      for (int g = 0; g < WR; ++g)
#pragma unroll
        for (int r = 0; r < R; ++r) sum[f][g][r] = 0;
    for (int c = lane * V; c < k_dim; c += MI_WAVE * V) {
      alignas(16) T wv[FW][WR][V];
#pragma unroll
      for (int f = 0; f < FW; ++f)
#pragma unroll
        for (int g = 0; g < WR; ++g) {
          const int row = min(f0 + f, features - 1) + g * features;  // (past the end: the last feature again, not written)
          // (the weights are read once: non-temporal, whole 16-byte pieces)
          *reinterpret_cast<int32x4_t*>(wv[f][g]) =
              __builtin_nontemporal_load(reinterpret_cast<const int32x4_t*>(w + (int64_t)row * k_dim + c));
        }
#pragma unroll
      for (int r = 0; r < R; ++r) {
        alignas(16) T xv[V];
        *reinterpret_cast<uint4*>(xv) = *reinterpret_cast<const uint4*>(rows + (size_t)r * k_dim + c);
#pragma unroll
        for (int j = 0; j < V; ++j) {
          const A xj = (A)to_f32(xv[j]);
#pragma unroll
          for (int f = 0; f < FW; ++f)
#pragma unroll
            for (int g = 0; g < WR; ++g) sum[f][g][r] += (A)to_f32(wv[f][g][j]) * xj;
        }
      }
    }
#pragma unroll
    for (int f = 0; f < FW; ++f)
#pragma unroll
      for (int r = 0; r < R; ++r) {
        A a = lanes_total(sum[f][0][r]);
        A b = GATED ? lanes_total(sum[f][WR - 1][r]) : (A)0;
        if (lane == 0 && r < n && f0 + f < features) {
          const int pair = listed[chunk + r];
          const A pw = MODE == EXPERT_SQUARED_RELU && pair_weight != nullptr ? (A)pair_weight[pair] : (A)1;
          out[(int64_t)pair * out_stride + f0 + f] = expert_feature<T, MODE, A>(a, b, pw);
        }
      }
  }
}

// The same for bfloat16 on the matrix cores (MFMA 16x16x32): a block owns one expert and 16 of its
// output features and takes the expert's listed pairs 16 rows at a time.  Its four waves share K (wave w
// takes the w-th quarter of the steps of 32 elements); per step a lane reads 16 bytes of weight row `lane % 16` and
// 16 bytes of pair `lane % 16`'s input row (both at elements 32 * step + 8 * (lane / 16)), which are the
// two operands as they are, so nothing is staged; rows past the expert's last pair read nothing.  The
// waves' sums meet in LDS in wave order, and lane (quad, col) of wave 0 writes features 4 * quad .. + 3 of
// pair col.  Needs K a multiple of 32.
typedef float f32x4_e __attribute__((ext_vector_type(4)));

template <int MODE>
__global__ __launch_bounds__(256) void expert_rows_mfma_kernel(
    const bf16_t* __restrict__ src, int64_t src_stride, int src_div, const bf16_t* __restrict__ weight,
    int64_t expert_stride, const int* __restrict__ listed, const int* __restrict__ first,
    const float* __restrict__ pair_weight, bf16_t* __restrict__ out, int64_t out_stride, int k_dim, int features) {
  constexpr bool GATED = MODE == EXPERT_SILU_GATED;
  __shared__ f32x4_e meet[GATED ? 2 : 1][3][MI_WAVE];
  const int e = blockIdx.y;  // (feature tiles run fastest: a chosen expert's blocks follow one another and spread over all XCDs)
  const int begin = first[e], end = first[e + 1];
  if (begin >= end) return;  // nobody chose this expert (the whole block leaves)
  const int wave = threadIdx.x / MI_WAVE, lane = threadIdx.x % MI_WAVE;
  const int col = lane % 16, quad = lane / 16;
  const int f0 = blockIdx.x * 16;
  const int my_feature = min(f0 + col, features - 1);  // (past the end: the last feature again, not written)
  const bf16_t* w_gate = weight + (int64_t)e * expert_stride + (int64_t)my_feature * k_dim + quad * 8;
  const bf16_t* w_up = w_gate + (int64_t)features * k_dim;
  const int steps = k_dim / 32;
  for (int chunk = begin; chunk < end; chunk += 16) {
    const int n = min(16, end - chunk);
    const int pair = col < n ? listed[chunk + col] : -1;
    // (lanes past the expert's last pair read the chunk's first row and count it as nothing)
    const bf16_t* x_row = src + (int64_t)((pair >= 0 ? pair : listed[chunk]) / src_div) * src_stride + quad * 8;
    f32x4_e acc_g = {0.f, 0.f, 0.f, 0.f}, acc_u = {0.f, 0.f, 0.f, 0.f};
    const bf16x8_t nothing = {};
    // a wave's quarter of K in one stretch (its consecutive loads then use whole cache lines), four
    // steps' loads asked for before the first of them is used
    const int lo = steps * wave / 4, hi = steps * (wave + 1) / 4;
    int step = lo;
    for (; step + 4 <= hi; step += 4) {
      bf16x8_t a_g[4], a_u[4], b[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        a_g[i] = *reinterpret_cast<const bf16x8_t*>(w_gate + (step + i) * 32);
        if constexpr (GATED) a_u[i] = *reinterpret_cast<const bf16x8_t*>(w_up + (step + i) * 32);
        b[i] = *reinterpret_cast<const bf16x8_t*>(x_row + (step + i) * 32);
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const bf16x8_t seen = pair >= 0 ? b[i] : nothing;
        acc_g = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a_g[i], seen, acc_g, 0, 0, 0);
        if constexpr (GATED) acc_u = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a_u[i], seen, acc_u, 0, 0, 0);
      }
    }
    for (; step < hi; ++step) {
      const bf16x8_t a_g = *reinterpret_cast<const bf16x8_t*>(w_gate + step * 32);
      const bf16x8_t got = *reinterpret_cast<const bf16x8_t*>(x_row + step * 32);
      const bf16x8_t seen = pair >= 0 ? got : nothing;
      acc_g = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a_g, seen, acc_g, 0, 0, 0);
      if constexpr (GATED) {
        const bf16x8_t a_u = *reinterpret_cast<const bf16x8_t*>(w_up + step * 32);
        acc_u = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a_u, seen, acc_u, 0, 0, 0);
      }
    }
    __syncthreads();  // (the last chunk's sums have been read)
    if (wave > 0) {
      meet[0][wave - 1][lane] = acc_g;
      if constexpr (GATED) meet[1][wave - 1][lane] = acc_u;
    }
    __syncthreads();
    if (wave == 0 && pair >= 0) {
#pragma unroll
      for (int w = 0; w < 3; ++w) {
        acc_g += meet[0][w][lane];
        if constexpr (GATED) acc_u += meet[1][w][lane];
      }
      bf16_t* o = out + (int64_t)pair * out_stride;
      const float pw = MODE == EXPERT_SQUARED_RELU && pair_weight != nullptr ? pair_weight[pair] : 1.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int f = f0 + 4 * quad + r;
        if (f < features) o[f] = expert_feature<bf16_t, MODE, float>(acc_g[r], acc_u[r], pw);
      }
    }
  }
}

// Many rows an expert (a prompt): a block owns one expert and 64 of its output features, a wave 16 of
// them over all of K, and the expert's listed pairs are taken 64 rows a pass: per step of 32 elements a wave
// reads its 16 weight rows once (16 bytes a lane) and the four row tiles' input rows (the same for the
// block's four waves, so three of four reads hit the cache), and makes 4 (gated: 8) MFMA 16x16x32.  An
// expert's weights are read once per 64 of its rows and its rows once per 64 of its features.
template <int MODE>
__global__ __launch_bounds__(256) void expert_tiles_mfma_kernel(
    const bf16_t* __restrict__ src, int64_t src_stride, int src_div, const bf16_t* __restrict__ weight,
    int64_t expert_stride, const int* __restrict__ listed, const int* __restrict__ first,
    const float* __restrict__ pair_weight, bf16_t* __restrict__ out, int64_t out_stride, int k_dim, int features) {
  constexpr bool GATED = MODE == EXPERT_SILU_GATED;
  constexpr int RT = 4;  // row tiles of 16
  const int e = blockIdx.y;
  const int begin = first[e], end = first[e + 1];
  if (begin >= end) return;
  const int wave = threadIdx.x / MI_WAVE, lane = threadIdx.x % MI_WAVE;
  const int col = lane % 16, quad = lane / 16;
  const int f0 = blockIdx.x * 64 + wave * 16;
  if (f0 >= features) return;  // (no barrier below: a wave past the last feature may leave)
  const int my_feature = min(f0 + col, features - 1);
  const bf16_t* w_gate = weight + (int64_t)e * expert_stride + (int64_t)my_feature * k_dim + quad * 8;
  const bf16_t* w_up = w_gate + (int64_t)features * k_dim;
  const int steps = k_dim / 32;
  const bf16x8_t nothing = {};
  for (int chunk = begin; chunk < end; chunk += 16 * RT) {
    const int n = min(16 * RT, end - chunk);
    int pair[RT];
    const bf16_t* x_row[RT];
#pragma unroll
    for (int t = 0; t < RT; ++t) {
      pair[t] = 16 * t + col < n ? listed[chunk + 16 * t + col] : -1;
      x_row[t] = src + (int64_t)((pair[t] >= 0 ? pair[t] : listed[chunk]) / src_div) * src_stride + quad * 8;
    }
    f32x4_e acc_g[RT], acc_u[RT];
#pragma unroll
    for (int t = 0; t < RT; ++t) acc_g[t] = acc_u[t] = f32x4_e{0.f, 0.f, 0.f, 0.f};
    auto one_step = [&](int step) {
      const bf16x8_t a_g = *reinterpret_cast<const bf16x8_t*>(w_gate + step * 32);
      bf16x8_t a_u = nothing;
      if constexpr (GATED) a_u = *reinterpret_cast<const bf16x8_t*>(w_up + step * 32);
      bf16x8_t b[RT];
#pragma unroll
      for (int t = 0; t < RT; ++t) b[t] = *reinterpret_cast<const bf16x8_t*>(x_row[t] + step * 32);
#pragma unroll
      for (int t = 0; t < RT; ++t) {
        if (16 * t >= n) continue;  // (a tile without rows: the same for the whole block)
        const bf16x8_t seen = pair[t] >= 0 ? b[t] : nothing;
        acc_g[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a_g, seen, acc_g[t], 0, 0, 0);
        if constexpr (GATED) acc_u[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a_u, seen, acc_u[t], 0, 0, 0);
      }
    };
    int step = 0;
    for (; step + 2 <= steps; step += 2) {
      one_step(step);
      one_step(step + 1);
    }
    for (; step < steps; ++step) one_step(step);
#pragma unroll
    for (int t = 0; t < RT; ++t) {
      if (pair[t] < 0) continue;
      bf16_t* o = out + (int64_t)pair[t] * out_stride;
      const float pw = MODE == EXPERT_SQUARED_RELU && pair_weight != nullptr ? pair_weight[pair[t]] : 1.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int f = f0 + 4 * quad + r;
        if (f < features) o[f] = expert_feature<bf16_t, MODE, float>(acc_g[t][r], acc_u[t][r], pw);
      }
    }
  }
}

template <typename T>
__global__ __launch_bounds__(256) void weighted_squared_relu_kernel(const T* __restrict__ z, int64_t z_stride,
                                                                    const float* __restrict__ weight, T* __restrict__ out,
                                                                    int64_t out_stride, int width) {
  using A = typename SumOf<T>::type;
  const int row = blockIdx.x, i = blockIdx.y * blockDim.x + threadIdx.x;
  if (i >= width) return;
  out[(int64_t)row * out_stride + i] =
      expert_feature<T, EXPERT_SQUARED_RELU, A>((A)to_f32(z[(int64_t)row * z_stride + i]), (A)0, (A)weight[row]);
}

}  // namespace

extern "C" int mi_route_top_k(int dtype, const void* x, int64_t x_stride, const float* router, const float* correction,
                              const float* gate_row, int* chosen, float* weights, float* shared_gate, int num_tokens,
                              int width, int outputs, int top, float route_scale, int scores, hipStream_t stream) {
  MI_REQUIRE(num_tokens >= 0 && width > 0 && x_stride >= width, "route_top_k: bad sizes tokens=%d width=%d", num_tokens, width);
  MI_REQUIRE(outputs > 0 && outputs <= MI_ROUTER_MAX_OUTPUTS && top > 0 && top <= outputs,
             "route_top_k: %d router outputs (at most %d) of which %d are chosen", outputs, MI_ROUTER_MAX_OUTPUTS, top);
  MI_REQUIRE(scores >= SCORES_SOFTMAX && scores <= SCORES_CHOSEN_SOFTMAX, "route_top_k: unknown scores %d", scores);
  MI_REQUIRE(gate_row == nullptr || shared_gate != nullptr, "route_top_k: a gate row needs a place for the gates");
  MI_REQUIRE(dtype == MI_F32 || dtype == MI_BF16, "route_top_k: unknown dtype %d", dtype);
  if (num_tokens == 0) return MI_OK;
  // as many tokens a block as fit its staging (rows in the element type, sums beside them), at most 4
  const size_t elem = dtype == MI_F32 ? 4 : 2, acc = dtype == MI_F32 ? 8 : 4;
  auto lds_for = [&](int r) { return (size_t)r * (outputs + 1) * acc + (size_t)r * width * elem; };
  const int per_block = lds_for(4) <= 64 * 1024 ? 4 : (lds_for(2) <= 64 * 1024 ? 2 : 1);
  MI_REQUIRE(lds_for(per_block) <= 64 * 1024, "route_top_k: rows of %d do not fit the block's staging", width);
  const int threads = num_tokens <= 64 ? 1024 : 256;
  const int blocks = ceil_div(num_tokens, per_block);
#define MI_ROUTE(T, R)                                                                                               \
  route_top_k_kernel<T, R><<<blocks, threads, lds_for(R), stream>>>((const T*)x, x_stride, router, correction, gate_row, \
                                                                    chosen, weights, shared_gate, num_tokens, width,    \
                                                                    outputs, top, route_scale, scores)
  if (dtype == MI_F32) {
    if (per_block == 4) MI_ROUTE(float, 4);
    else if (per_block == 2) MI_ROUTE(float, 2);
    else MI_ROUTE(float, 1);
  } else {
    if (per_block == 4) MI_ROUTE(bf16_t, 4);
    else if (per_block == 2) MI_ROUTE(bf16_t, 2);
    else MI_ROUTE(bf16_t, 1);
  }
#undef MI_ROUTE
  MI_CHECK_LAUNCH("route_top_k");
  return MI_OK;
}

// act: [num_tokens * top, ff]; rows of pairs whose expert is an identity expert are not written.  mode: 1 silu
// gated, 2 squared relu of the weighted product (pair_weight float32 [num_tokens * top] or null: 1).
extern "C" int mi_expert_gate_up(int dtype, int mode, const void* x, int64_t x_stride, const void* gate_up, const int* chosen,
                                 const float* pair_weight, void* act, int num_tokens, int width, int ff, int experts,
                                 int top, hipStream_t stream) {
  MI_REQUIRE(num_tokens >= 0 && width > 0 && ff > 0 && experts > 0 && top > 0 && x_stride >= width,
             "expert_gate_up: bad sizes tokens=%d width=%d ff=%d experts=%d top=%d", num_tokens, width, ff, experts, top);
  MI_REQUIRE(dtype == MI_F32 || dtype == MI_BF16, "expert_gate_up: unknown dtype %d", dtype);
  MI_REQUIRE(mode == EXPERT_SILU_GATED || (mode == EXPERT_SQUARED_RELU), "expert_gate_up: mode %d", mode);
  const size_t lds = (size_t)width * (dtype == MI_F32 ? 4 : 2);
  MI_REQUIRE(lds <= 64 * 1024, "expert_gate_up: rows of %d do not fit the block's staging", width);
  MI_REQUIRE((int64_t)num_tokens * top <= 0x7fffffff / 2 && ceil_div(ff, MI_EXPERT_FEATURES) <= 65535, "expert_gate_up: too many pairs or features");
  if (num_tokens == 0) return MI_OK;
  dim3 grid(num_tokens * top, ceil_div(ff, MI_EXPERT_FEATURES));
#define MI_GATE_UP(T, MODE)                                                                                              \
  expert_gate_up_kernel<T, MODE><<<grid, 256, lds, stream>>>((const T*)x, x_stride, (const T*)gate_up, chosen, pair_weight, \
                                                             (T*)act, width, ff, experts, top)
  if (dtype == MI_F32) {
    if (mode == EXPERT_SILU_GATED) MI_GATE_UP(float, EXPERT_SILU_GATED);
    else MI_GATE_UP(float, EXPERT_SQUARED_RELU);
  } else {
    if (mode == EXPERT_SILU_GATED) MI_GATE_UP(bf16_t, EXPERT_SILU_GATED);
    else MI_GATE_UP(bf16_t, EXPERT_SQUARED_RELU);
  }
#undef MI_GATE_UP
  MI_CHECK_LAUNCH("expert_gate_up");
  return MI_OK;
}

extern "C" int mi_expert_down_combine(int dtype, const void* act, const void* down, const int* chosen, const float* weights,
                                      const void* x, int64_t x_stride, const void* shared, int64_t shared_stride,
                                      const float* shared_gate, void* out, int num_tokens, int width, int ff, int experts,
                                      int top, hipStream_t stream) {
  MI_REQUIRE(num_tokens >= 0 && width > 0 && ff > 0 && experts > 0 && top > 0 && x_stride >= width,
             "expert_down_combine: bad sizes tokens=%d width=%d ff=%d experts=%d top=%d", num_tokens, width, ff, experts, top);
  MI_REQUIRE(shared == nullptr || shared_stride >= width, "expert_down_combine: a shared expert's rows are shorter than a row");
  MI_REQUIRE(dtype == MI_F32 || dtype == MI_BF16, "expert_down_combine: unknown dtype %d", dtype);
  const size_t lds = (size_t)top * ff * (dtype == MI_F32 ? 4 : 2);
  MI_REQUIRE(lds <= 64 * 1024, "expert_down_combine: %d rows of %d do not fit the block's staging", top, ff);
  MI_REQUIRE(ceil_div(width, MI_EXPERT_FEATURES) <= 65535, "expert_down_combine: too many columns");
  if (num_tokens == 0) return MI_OK;
  dim3 grid(num_tokens, ceil_div(width, MI_EXPERT_FEATURES));
  if (dtype == MI_F32)
    expert_down_combine_kernel<float><<<grid, 256, lds, stream>>>(
        (const float*)act, (const float*)down, chosen, weights, (const float*)x, x_stride, (const float*)shared, shared_stride,
        shared_gate, (float*)out, width, ff, experts, top);
  else
    expert_down_combine_kernel<bf16_t><<<grid, 256, lds, stream>>>(
        (const bf16_t*)act, (const bf16_t*)down, chosen, weights, (const bf16_t*)x, x_stride, (const bf16_t*)shared,
        shared_stride, shared_gate, (bf16_t*)out, width, ff, experts, top);
  MI_CHECK_LAUNCH("expert_down_combine");
  return MI_OK;
}

// made: rows of expert outputs [*, width]; pair (t, k) finds its row at where[t * top + k] (or at
// t * top + k itself with where = null).
extern "C" int mi_expert_combine(int dtype, const void* made, const int* where, const int* chosen, const float* weights,
                                 const void* x, int64_t x_stride, const void* shared, int64_t shared_stride,
                                 const float* shared_gate, void* out, int num_tokens, int width, int experts, int top,
                                 hipStream_t stream) {
  MI_REQUIRE(num_tokens >= 0 && width > 0 && experts > 0 && top > 0 && x_stride >= width,
             "expert_combine: bad sizes tokens=%d width=%d experts=%d top=%d", num_tokens, width, experts, top);
  MI_REQUIRE(shared == nullptr || shared_stride >= width, "expert_combine: a shared expert's rows are shorter than a row");
  MI_REQUIRE(dtype == MI_F32 || dtype == MI_BF16, "expert_combine: unknown dtype %d", dtype);
  if (num_tokens == 0) return MI_OK;
  const bool vec = width % 4 == 0 && x_stride % 4 == 0 && shared_stride % 4 == 0 && is_aligned16(made) && is_aligned16(x) &&
                   is_aligned16(shared) && is_aligned16(out);
#define MI_COMBINE(T, VEC)                                                                                              \
  expert_combine_kernel<T, VEC><<<num_tokens, 256, 0, stream>>>((const T*)made, where, chosen, weights, (const T*)x,    \
                                                                x_stride, (const T*)shared, shared_stride, shared_gate, \
                                                                (T*)out, width, experts, top)
  if (dtype == MI_F32) {
    if (vec) MI_COMBINE(float, 4);
    else MI_COMBINE(float, 1);
  } else {
    if (vec) MI_COMBINE(bf16_t, 4);
    else MI_COMBINE(bf16_t, 1);
  }
#undef MI_COMBINE
  MI_CHECK_LAUNCH("expert_combine");
  return MI_OK;
}

extern "C" int mi_expert_sort(const int* chosen, int* listed, int* first, int pairs, int experts, hipStream_t stream) {
  MI_REQUIRE(pairs >= 0 && experts > 0 && experts <= MI_SORT_MAX_EXPERTS, "expert_sort: %d pairs over %d experts (at most %d)", pairs,
             experts, MI_SORT_MAX_EXPERTS);
  expert_sort_kernel<<<1, pairs > 256 ? 1024 : 256, 0, stream>>>(chosen, listed, first, pairs, experts);
  MI_CHECK_LAUNCH("expert_sort");
  return MI_OK;
}

// Whether mi_route_few takes a step of these sizes (bfloat16 only).
extern "C" int mi_route_few_takes(int num_tokens, int width, int outputs, int top) {
  return num_tokens > 0 && num_tokens <= MI_ROUTE_FEW_TOKENS && num_tokens * top <= MI_ROUTE_FEW_PAIRS && width >= 4 && width % 4 == 0 &&
         outputs > 0 && outputs <= MI_ROUTER_MAX_OUTPUTS;
}

// mi_route_top_k and mi_expert_sort for few bfloat16 tokens in two launches; `logits`: scratch
// [num_tokens, outputs + (gate row ? 1 : 0)] floats.
extern "C" int mi_route_few(const void* x, int64_t x_stride, const float* router, const float* correction, const float* gate_row,
                            float* logits, int* chosen, float* weights, float* shared_gate, int* listed, int* first,
                            int num_tokens, int width, int outputs, int experts, int top, float route_scale, int scores,
                            hipStream_t stream) {
  MI_REQUIRE(mi_route_few_takes(num_tokens, width, outputs, top) && x_stride >= width && x_stride % 4 == 0 && (uintptr_t)x % 8 == 0 &&
                 is_aligned16(router) && is_aligned16(gate_row),
             "route_few: %d tokens of %d columns, %d outputs", num_tokens, width, outputs);
  MI_REQUIRE(top > 0 && top <= outputs && experts > 0 && experts <= outputs, "route_few: %d of %d outputs, %d experts", top, outputs, experts);
  MI_REQUIRE(scores >= SCORES_SOFTMAX && scores <= SCORES_CHOSEN_SOFTMAX, "route_few: unknown scores %d", scores);
  MI_REQUIRE(gate_row == nullptr || shared_gate != nullptr, "route_few: a gate row needs a place for the gates");
  const int total = outputs + (gate_row != nullptr ? 1 : 0);
  route_logits_kernel<<<dim3(total, ceil_div(num_tokens, 8)), 256, 0, stream>>>((const bf16_t*)x, x_stride, router, gate_row, logits,
                                                                               num_tokens, width, outputs, total);
  MI_CHECK_LAUNCH("route_logits");
  const int threads = min(1024, num_tokens * MI_WAVE);
  route_list_kernel<<<1, threads, (size_t)(threads / MI_WAVE) * outputs * 4, stream>>>(
      logits, correction, chosen, weights, shared_gate, listed, first, num_tokens, outputs, total, experts, top, route_scale, scores);
  MI_CHECK_LAUNCH("route_list");
  return MI_OK;
}

// Rows a block keeps in LDS at a time for rows of k_dim elements (0: such rows do not fit).
extern "C" int mi_expert_rows_at_once(int dtype, int k_dim) {
  const size_t row = (size_t)k_dim * (dtype == MI_F32 ? 4 : 2);
  if (dtype != MI_F32 && 8 * row <= 64 * 1024) return 8;
  if (4 * row <= 64 * 1024) return 4;
  if (2 * row <= 64 * 1024) return 2;
  return 0;
}

// mode 1 (silu gated): weight [experts, 2 * features, k_dim], out[pair, f] = silu(gate_f . row) * (up_f . row) with
// the row of pair p at src[p / src_div]; mode 2: weight [experts, features, k_dim], out[pair, f] =
// relu(pair_weight[pair] * (w_f . row))^2 (pair_weight null: 1); mode 0: out[pair, f] = w_f . row.
// many_rows = 1 (bfloat16 with k_dim a multiple of 32 only): blocks of 64 features that take 64 rows a pass.
extern "C" int mi_expert_rows(int dtype, int mode, const void* src, int64_t src_stride, int src_div, const void* weight,
                              const int* listed, const int* first, const float* pair_weight, void* out, int64_t out_stride,
                              int experts, int k_dim, int features, int many_rows, hipStream_t stream) {
  MI_REQUIRE(experts > 0 && experts <= 65535 && k_dim > 0 && features > 0 && src_div > 0 && src_stride >= k_dim && out_stride >= features,
             "expert_rows: bad sizes experts=%d k=%d features=%d", experts, k_dim, features);
  MI_REQUIRE(dtype == MI_F32 || dtype == MI_BF16, "expert_rows: unknown dtype %d", dtype);
  MI_REQUIRE(mode == EXPERT_PLAIN || mode == EXPERT_SILU_GATED || (mode == EXPERT_SQUARED_RELU),
             "expert_rows: mode %d", mode);
  const int elem = dtype == MI_F32 ? 4 : 2, step = 16 / elem;
  MI_REQUIRE(k_dim % step == 0 && src_stride % step == 0 && is_aligned16(src) && is_aligned16(weight),
             "expert_rows: rows of %d elements are not read 16 bytes at a time", k_dim);
  const int64_t expert_stride = (int64_t)(mode == EXPERT_SILU_GATED ? 2 : 1) * features * k_dim;
  dim3 grid(ceil_div(features, 16), experts);
#define MI_BY_MODE(LAUNCH)                                   \
  do {                                                       \
    if (mode == EXPERT_SILU_GATED) LAUNCH(EXPERT_SILU_GATED); \
    else if (mode == EXPERT_SQUARED_RELU) LAUNCH(EXPERT_SQUARED_RELU); \
    else LAUNCH(EXPERT_PLAIN);                               \
  } while (0)
  if (dtype == MI_BF16 && k_dim % 32 == 0) {  // the matrix cores
    dim3 tiles(ceil_div(features, 64), experts);
#define MI_TILES(MODE)                                                                                              \
  expert_tiles_mfma_kernel<MODE><<<tiles, 256, 0, stream>>>((const bf16_t*)src, src_stride, src_div, (const bf16_t*)weight, \
                                                            expert_stride, listed, first, pair_weight, (bf16_t*)out,  \
                                                            out_stride, k_dim, features)
#define MI_MFMA(MODE)                                                                                               \
  expert_rows_mfma_kernel<MODE><<<grid, 256, 0, stream>>>((const bf16_t*)src, src_stride, src_div, (const bf16_t*)weight, \
                                                          expert_stride, listed, first, pair_weight, (bf16_t*)out,    \
                                                          out_stride, k_dim, features)
    if (many_rows) MI_BY_MODE(MI_TILES);
    else MI_BY_MODE(MI_MFMA);
#undef MI_TILES
#undef MI_MFMA
    MI_CHECK_LAUNCH("expert_rows_mfma");
    return MI_OK;
  }
  const int at_once = mi_expert_rows_at_once(dtype, k_dim);
  MI_REQUIRE(at_once > 0, "expert_rows: rows of %d do not fit the block's staging", k_dim);
  const size_t lds = (size_t)at_once * k_dim * elem;
#define MI_ROWS_OF(T, R, MODE)                                                                                    \
  expert_rows_kernel<T, R, MODE><<<grid, 256, lds, stream>>>((const T*)src, src_stride, src_div, (const T*)weight, \
                                                             expert_stride, listed, first, pair_weight, (T*)out,   \
                                                             out_stride, k_dim, features)
#define MI_ROWS_F4(MODE) MI_ROWS_OF(float, 4, MODE)
#define MI_ROWS_F2(MODE) MI_ROWS_OF(float, 2, MODE)
#define MI_ROWS_B8(MODE) MI_ROWS_OF(bf16_t, 8, MODE)
#define MI_ROWS_B4(MODE) MI_ROWS_OF(bf16_t, 4, MODE)
#define MI_ROWS_B2(MODE) MI_ROWS_OF(bf16_t, 2, MODE)
  if (dtype == MI_F32) {
    if (at_once == 4) MI_BY_MODE(MI_ROWS_F4);
    else MI_BY_MODE(MI_ROWS_F2);
  } else {
    if (at_once == 8) MI_BY_MODE(MI_ROWS_B8);
    else if (at_once == 4) MI_BY_MODE(MI_ROWS_B4);
    else MI_BY_MODE(MI_ROWS_B2);
  }
#undef MI_ROWS_OF
#undef MI_ROWS_F4
#undef MI_ROWS_F2
#undef MI_ROWS_B8
#undef MI_ROWS_B4
#undef MI_ROWS_B2
#undef MI_BY_MODE
  MI_CHECK_LAUNCH("expert_rows");
  return MI_OK;
}

// out[row, f] = relu(z * weight[row])^2 for rows of a product made by others (row stride z_stride).
extern "C" int mi_weighted_squared_relu(int dtype, const void* z, int64_t z_stride, const float* weight, void* out,
                                        int64_t out_stride, int num_rows, int width, hipStream_t stream) {
  MI_REQUIRE(num_rows >= 0 && width > 0 && z_stride >= width && out_stride >= width, "weighted_squared_relu: bad sizes rows=%d width=%d",
             num_rows, width);
  MI_REQUIRE(ceil_div(width, 256) <= 65535, "weighted_squared_relu: width %d is too large", width);
  MI_REQUIRE(dtype == MI_F32 || dtype == MI_BF16, "weighted_squared_relu: unknown dtype %d", dtype);
  if (num_rows == 0) return MI_OK;
  dim3 grid(num_rows, ceil_div(width, 256));
  if (dtype == MI_F32)
    weighted_squared_relu_kernel<float><<<grid, 256, 0, stream>>>((const float*)z, z_stride, weight, (float*)out, out_stride, width);
  else
    weighted_squared_relu_kernel<bf16_t><<<grid, 256, 0, stream>>>((const bf16_t*)z, z_stride, weight, (bf16_t*)out, out_stride, width);
  MI_CHECK_LAUNCH("weighted_squared_relu");
  return MI_OK;
}
