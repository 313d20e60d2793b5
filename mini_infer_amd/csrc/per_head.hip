// A product head by head: out[t, h, n] = sum_k x[t, h, k] * w[h, n, k]  (times logistic(gate[t, h, n])
// where a gate is given), bfloat16 with float32 sums: the maps of a latent attention layer that are
// folded into its queries and applied behind its attention.
//
// MFMA 16x16x32 with weight rows as the first operand and tokens as the second: per step of 32 elements
// a lane reads 16 bytes of weight row `lane % 16` and 16 bytes of token `lane % 16` (both at elements
// 32 * step + 8 * (lane / 16)), which are the operands as they are.  A block owns one head.
//   SHARE  up to 64 tokens: the block owns 16 features and its four waves share K (their sums meet in LDS in
//          wave order), so that even a short K keeps every wave busy with one stretch of weights.
//   else   a wave owns 16 features over all of K and RT row tiles of 16 tokens share each weight operand.
// K is a multiple of 8; what a last, shorter step lacks counts as zero on both sides.
#include "common.h"

namespace {

typedef float f32x4_h __attribute__((ext_vector_type(4)));

struct PerHeadShape {
  int64_t x_stride, x_head, w_head, out_stride, out_head, gate_stride, gate_head;
  int tokens, k_dim, features;
};

__device__ __forceinline__ void put_features(bf16_t* __restrict__ out, const bf16_t* __restrict__ gate, const PerHeadShape& s,
                                             int h, int t, int f0, const f32x4_h& sum) {
  bf16_t* o = out + (int64_t)t * s.out_stride + h * s.out_head;
  const bf16_t* g = gate != nullptr ? gate + (int64_t)t * s.gate_stride + h * s.gate_head : nullptr;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int f = f0 + r;
    if (f >= s.features) continue;
    float v = sum[r];
    // (the product as the element type holds it, then the gate)
    if (g != nullptr) v = to_f32(from_f32<bf16_t>(v)) * mi_logistic(to_f32(g[f]));
    o[f] = from_f32<bf16_t>(v);
  }
}

template <int RT, bool SHARE>
__global__ __launch_bounds__(256) void per_head_kernel(const bf16_t* __restrict__ x, const bf16_t* __restrict__ w,
                                                       const bf16_t* __restrict__ gate, bf16_t* __restrict__ out,
                                                       PerHeadShape s) {
  __shared__ f32x4_h meet[SHARE ? 3 : 1][RT][MI_WAVE];
  const int h = blockIdx.y, t0 = blockIdx.z * 16 * RT;
  const int wave = threadIdx.x / MI_WAVE, lane = threadIdx.x % MI_WAVE;
  const int col = lane % 16, quad = lane / 16;
  const int f0 = SHARE ? blockIdx.x * 16 : blockIdx.x * 64 + wave * 16;
  if (f0 >= s.features) return;  // (SHARE: the whole block; else: no barrier below)
  const bf16_t* w_row = w + (int64_t)h * s.w_head + (int64_t)min(f0 + col, s.features - 1) * s.k_dim + quad * 8;
  const bf16_t* x_row[RT];
#pragma unroll
  for (int i = 0; i < RT; ++i)  // (tokens past the last one read it again; their sums are not written)
    x_row[i] = x + (int64_t)min(t0 + 16 * i + col, s.tokens - 1) * s.x_stride + h * s.x_head + quad * 8;
  f32x4_h acc[RT];
#pragma unroll
  for (int i = 0; i < RT; ++i) acc[i] = f32x4_h{0.f, 0.f, 0.f, 0.f};
  const int steps = (s.k_dim + 31) / 32;
  const int lo = SHARE ? steps * wave / 4 : 0, hi = SHARE ? steps * (wave + 1) / 4 : steps;
  const bf16x8_t nothing = {};
  // whole steps, four at a time (their loads are asked for before the first is used), then the rest
  const int whole = min(hi, s.k_dim / 32);
  int step = lo;
  for (; step + 4 <= whole; step += 4) {
    bf16x8_t a[4], b[4][RT];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      a[j] = *reinterpret_cast<const bf16x8_t*>(w_row + (step + j) * 32);
#pragma unroll
      for (int i = 0; i < RT; ++i) b[j][i] = *reinterpret_cast<const bf16x8_t*>(x_row[i] + (step + j) * 32);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
      for (int i = 0; i < RT; ++i) acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[j], b[j][i], acc[i], 0, 0, 0);
  }
  for (; step < hi; ++step) {
    const bool there = step * 32 + quad * 8 < s.k_dim;
    const bf16x8_t a = there ? *reinterpret_cast<const bf16x8_t*>(w_row + step * 32) : nothing;
#pragma unroll
    for (int i = 0; i < RT; ++i) {
      const bf16x8_t b = there ? *reinterpret_cast<const bf16x8_t*>(x_row[i] + step * 32) : nothing;
      acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, acc[i], 0, 0, 0);
    }
  }
  if constexpr (SHARE) {
    if (wave > 0) {
#pragma unroll
      for (int i = 0; i < RT; ++i) meet[wave - 1][i][lane] = acc[i];
    }
    __syncthreads();
    if (wave > 0) return;
#pragma unroll
    for (int other = 0; other < 3; ++other)
#pragma unroll
      for (int i = 0; i < RT; ++i) acc[i] += meet[other][i][lane];
  }
#pragma unroll
  for (int i = 0; i < RT; ++i) {
    const int t = t0 + 16 * i + col;
    if (t < s.tokens) put_features(out, gate, s, h, t, f0 + 4 * quad, acc[i]);
  }
}

}  // namespace

// x[t, h, k] at t * x_stride + h * x_head + k; w [heads, features, k_dim]; out (and gate, null: none) [t, h, n] at
// t * stride + h * head + n.  Strides in elements; k_dim, x_stride and x_head multiples of 8, x and w on 16 bytes.
extern "C" int mi_per_head_bf16(const void* x, int64_t x_stride, int64_t x_head, const void* w, const void* gate,
                                int64_t gate_stride, int64_t gate_head, void* out, int64_t out_stride, int64_t out_head,
                                int tokens, int heads, int k_dim, int features, hipStream_t stream) {
  MI_REQUIRE(tokens >= 0 && heads > 0 && heads <= 65535 && k_dim > 0 && features > 0, "per_head: bad sizes tokens=%d heads=%d k=%d features=%d",
             tokens, heads, k_dim, features);
  MI_REQUIRE(k_dim % 8 == 0 && x_stride % 8 == 0 && x_head % 8 == 0 && ((uintptr_t)x | (uintptr_t)w) % 16 == 0,
             "per_head: rows are read 16 bytes at a time (k=%d)", k_dim);
  if (tokens == 0) return MI_OK;
  const PerHeadShape s = {x_stride, x_head, (int64_t)features * k_dim, out_stride, out_head, gate_stride, gate_head, tokens, k_dim, features};
  if (tokens <= 16) {
    dim3 grid(ceil_div(features, 16), heads, 1);
    per_head_kernel<1, true><<<grid, 256, 0, stream>>>((const bf16_t*)x, (const bf16_t*)w, (const bf16_t*)gate, (bf16_t*)out, s);
  } else if (tokens <= 64) {
    dim3 grid(ceil_div(features, 16), heads, 1);
    if (tokens <= 32) per_head_kernel<2, true><<<grid, 256, 0, stream>>>((const bf16_t*)x, (const bf16_t*)w, (const bf16_t*)gate, (bf16_t*)out, s);
    else per_head_kernel<4, true><<<grid, 256, 0, stream>>>((const bf16_t*)x, (const bf16_t*)w, (const bf16_t*)gate, (bf16_t*)out, s);
  } else {
    MI_REQUIRE(ceil_div(tokens, 64) <= 65535, "per_head: too many tokens (%d)", tokens);
    dim3 grid(ceil_div(features, 64), heads, ceil_div(tokens, 64));
    per_head_kernel<4, false><<<grid, 256, 0, stream>>>((const bf16_t*)x, (const bf16_t*)w, (const bf16_t*)gate, (bf16_t*)out, s);
  }
  MI_CHECK_LAUNCH("per_head");
  return MI_OK;
}
