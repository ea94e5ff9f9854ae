// What a block's branches leave, added to the residual stream, and one or two RMS norms of the new stream, in one pass
// over a token's row:
//
//   v      = h[row] + (a + b + bias + sum_s topk_w[row, s] y[dest[row, s]] + gate[row] shared[row]) + again + step
//   h[row] = v (unless rows are picked);   out_i[r] = v * rsqrt(mean(v^2) + eps) * w_i
//
// Every term is optional: a, b dense results [T, width]; bias a vector (a last product's bias); the experts' sum with its
// shared expert (`shared_gate` null: weight 1); again: a row of a table times a number, row ids[row] of it (the embedding
// once more), or row `row` without ids; step a vector.  All sums are float32; the branches' own sum is formed first.
// Without norms (w1 null) only h is updated.
#include "common.h"

#define BN_MAX_K 32

struct BranchTerms {
  const void* a;
  const void* b;
  const void* bias;
  const void* y;
  const void* shared;
  const void* again;
  const void* step;
  const int32_t* dest;
  const float* topk_w;
  const float* shared_gate;
  const int32_t* ids;
  int64_t again_rows;
  float again_scale;
  int bias_dtype, again_dtype, step_dtype, k;
};

// Any element types and widths, one column at a time.  h is read twice when it is updated (every thread reads back what
// it wrote itself); with picked rows the sum is formed twice.
template <typename T>
__global__ void __launch_bounds__(1024)
branch_norm_kernel(float* __restrict__ h, BranchTerms m, const void* __restrict__ w1, int w1_dtype, T* __restrict__ out1,
                   const void* __restrict__ w2, int w2_dtype, T* __restrict__ out2, const int32_t* __restrict__ rows,
                   int64_t width, float eps) {
  __shared__ float red[16];
  __shared__ float sw[BN_MAX_K];
  __shared__ int32_t sd[BN_MAX_K];
  const int64_t r = blockIdx.x;
  const int64_t row = rows ? rows[r] : r;
  if (m.y && static_cast<int>(threadIdx.x) < m.k) {
    sw[threadIdx.x] = m.topk_w[row * m.k + threadIdx.x];
    sd[threadIdx.x] = m.dest[row * m.k + threadIdx.x];
  }
  __syncthreads();
  const float sg = m.shared_gate ? m.shared_gate[row] : 1.0f;
  const int64_t id = m.ids ? m.ids[row] : row;
  const bool again = m.again && id >= 0 && id < m.again_rows;
  float* hr = h + row * width;
  auto value = [&](int64_t c) {
    float d = 0.f;
    if (m.a) d += ix_load(static_cast<const T*>(m.a) + row * width + c);
    if (m.b) d += ix_load(static_cast<const T*>(m.b) + row * width + c);
    if (m.bias) d += ix_load_rt(m.bias, m.bias_dtype, c);
    if (m.y)
      for (int s = 0; s < m.k; ++s) d += sw[s] * ix_load(static_cast<const T*>(m.y) + static_cast<int64_t>(sd[s]) * width + c);
    if (m.shared) d += sg * ix_load(static_cast<const T*>(m.shared) + row * width + c);
    float v = hr[c] + d;
    if (again) v += ix_load_rt(m.again, m.again_dtype, id * width + c) * m.again_scale;
    if (m.step) v += ix_load_rt(m.step, m.step_dtype, c);
    return v;
  };
  float sumsq = 0.f;
  for (int64_t c = threadIdx.x; c < width; c += blockDim.x) {
    const float v = value(c);
    if (!rows) hr[c] = v;
    sumsq += v * v;
  }
  if (!w1) return;
  sumsq = ix_block_sum(sumsq, red);
  const float inv = 1.0f / sqrtf(sumsq / static_cast<float>(width) + eps);
  for (int64_t c = threadIdx.x; c < width; c += blockDim.x) {
    const float v = rows ? value(c) : hr[c];
    ix_store(out1 + r * width + c, v * inv * ix_load_rt(w1, w1_dtype, c));
    if (w2) ix_store(out2 + r * width + c, v * inv * ix_load_rt(w2, w2_dtype, c));
  }
}

__device__ __forceinline__ float4 bn_load4(const void* base, int dtype, int64_t i) {  // i a multiple of 4
  if (dtype == IX_F32) return *reinterpret_cast<const float4*>(static_cast<const float*>(base) + i);
  const uint2 p = *reinterpret_cast<const uint2*>(static_cast<const uint16_t*>(base) + i);
  return make_float4(__uint_as_float(p.x << 16), __uint_as_float(p.x & 0xffff0000u), __uint_as_float(p.y << 16),
                     __uint_as_float(p.y & 0xffff0000u));
}
__device__ __forceinline__ void bn_add4(float4& v, float f, const float4& d) {
  v.x += f * d.x;
  v.y += f * d.y;
  v.z += f * d.z;
  v.w += f * d.w;
}
__device__ __forceinline__ void bn_store4(uint16_t* dst, const float4& v, float inv, const float4& w) {
  uint2 o;
  o.x = ix_f32_to_bf16(v.x * inv * w.x) | static_cast<uint32_t>(ix_f32_to_bf16(v.y * inv * w.y)) << 16;
  o.y = ix_f32_to_bf16(v.z * inv * w.z) | static_cast<uint32_t>(ix_f32_to_bf16(v.w * inv * w.w)) << 16;
  *reinterpret_cast<uint2*>(dst) = o;
}

// bfloat16 with a width that is a multiple of 4: NV times four columns per thread, kept in registers between the sum of
// squares and the norms; what a column needs is asked for at once (the experts' rows eight at a time).
#define BN_SLOTS 8
template <int NV>
__global__ void __launch_bounds__(1024)
branch_norm_vec4_kernel(float* __restrict__ h, BranchTerms m, const void* __restrict__ w1, int w1_dtype,
                        uint16_t* __restrict__ out1, const void* __restrict__ w2, int w2_dtype, uint16_t* __restrict__ out2,
                        const int32_t* __restrict__ rows, int64_t width, float eps) {
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  const int64_t row = rows ? rows[r] : r;
  const float sg = m.shared_gate ? m.shared_gate[row] : 1.0f;
  const int64_t id = m.ids ? m.ids[row] : row;
  const bool again = m.again && id >= 0 && id < m.again_rows;
  float* hr = h + row * width;
  float4 v[NV];
  float4 wa[NV], wb[NV];
  float sumsq = 0.f;
#pragma unroll
  for (int u = 0; u < NV; ++u) {
    const int64_t c = 4 * (threadIdx.x + static_cast<int64_t>(u) * blockDim.x);
    v[u] = wa[u] = wb[u] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (c >= width) continue;
    const float4 old = *reinterpret_cast<const float4*>(hr + c);
    float4 d = make_float4(0.f, 0.f, 0.f, 0.f);
    if (m.y) {
      const int32_t* dest = m.dest + row * m.k;
      const float* weight = m.topk_w + row * m.k;
      for (int s0 = 0; s0 < m.k; s0 += BN_SLOTS) {
        float4 e[BN_SLOTS];
#pragma unroll
        for (int s = 0; s < BN_SLOTS; ++s)
          if (s0 + s < m.k) e[s] = bn_load4(m.y, IX_BF16, static_cast<int64_t>(dest[s0 + s]) * width + c);
#pragma unroll
        for (int s = 0; s < BN_SLOTS; ++s)
          if (s0 + s < m.k) bn_add4(d, weight[s0 + s], e[s]);
      }
    }
    if (m.a) bn_add4(d, 1.0f, bn_load4(m.a, IX_BF16, row * width + c));
    if (m.b) bn_add4(d, 1.0f, bn_load4(m.b, IX_BF16, row * width + c));
    if (m.bias) bn_add4(d, 1.0f, bn_load4(m.bias, m.bias_dtype, c));
    if (m.shared) bn_add4(d, sg, bn_load4(m.shared, IX_BF16, row * width + c));
    if (w1) wa[u] = bn_load4(w1, w1_dtype, c);
    if (w2) wb[u] = bn_load4(w2, w2_dtype, c);
    v[u] = make_float4(old.x + d.x, old.y + d.y, old.z + d.z, old.w + d.w);
    if (again) {
      const float4 t = bn_load4(m.again, m.again_dtype, id * width + c);
      bn_add4(v[u], m.again_scale, t);
    }
    if (m.step) bn_add4(v[u], 1.0f, bn_load4(m.step, m.step_dtype, c));
    if (!rows) *reinterpret_cast<float4*>(hr + c) = v[u];
    sumsq += v[u].x * v[u].x;
    sumsq += v[u].y * v[u].y;
    sumsq += v[u].z * v[u].z;
    sumsq += v[u].w * v[u].w;
  }
  if (!w1) return;
  sumsq = ix_block_sum(sumsq, red);
  const float inv = 1.0f / sqrtf(sumsq / static_cast<float>(width) + eps);
#pragma unroll
  for (int u = 0; u < NV; ++u) {
    const int64_t c = 4 * (threadIdx.x + static_cast<int64_t>(u) * blockDim.x);
    if (c >= width) continue;
    bn_store4(out1 + r * width + c, v[u], inv, wa[u]);
    if (w2) bn_store4(out2 + r * width + c, v[u], inv, wb[u]);
  }
}

// h float32 [T, width]; a, b, y, shared, out1, out2 of `dtype`; rows int32 [n_rows] or null (then n_rows = T).
extern "C" int ix_branch_norm(float* h, int dtype, const void* a, const void* b, const void* bias, int bias_dtype,
                              const void* y, const int32_t* dest, const float* topk_w, int k, const void* shared,
                              const float* shared_gate, const void* again, int again_dtype, const int32_t* ids,
                              int64_t again_rows, float again_scale, const void* step, int step_dtype, const void* w1,
                              int w1_dtype, void* out1, const void* w2, int w2_dtype, void* out2, const int32_t* rows,
                              int64_t n_rows, int64_t width, float eps, hipStream_t stream) {
  IX_REQUIRE(n_rows >= 0 && width > 0, "sizes must be positive");
  IX_REQUIRE(dtype == IX_F32 || dtype == IX_BF16, "dtype must be float32 or bfloat16");
  IX_REQUIRE(y == nullptr || (k > 0 && k <= BN_MAX_K && dest && topk_w), "between 1 and 32 experts per token, with their rows and weights");
  IX_REQUIRE((w1 == nullptr) == (out1 == nullptr) && (w2 == nullptr) == (out2 == nullptr) && (w1 || !w2),
             "a norm's weight and its result come together, the first norm's before the second's");
  IX_REQUIRE(rows == nullptr || w1 != nullptr, "picked rows are for a norm's result");
  for (const int d : {bias_dtype, again_dtype, step_dtype, w1_dtype, w2_dtype})
    IX_REQUIRE(d == IX_F32 || d == IX_BF16, "vectors and tables must be float32 or bfloat16");
  if (n_rows == 0) return 0;
  const BranchTerms m = {a, b, bias, y, shared, again, step, dest, topk_w, shared_gate, ids, again_rows, again_scale,
                         bias_dtype, again_dtype, step_dtype, k};
  uintptr_t at = 0;
  for (const void* p : {(const void*)h, a, b, bias, y, shared, again, step, w1, w2, (const void*)out1, (const void*)out2})
    at |= reinterpret_cast<uintptr_t>(p);
  const dim3 grid(static_cast<unsigned>(n_rows));
  if (dtype == IX_BF16 && width % 4 == 0 && width <= 4 * 4096 && (at & 15) == 0) {
    const int threads = static_cast<int>(std::min<int64_t>(1024, (width / 4 + 63) / 64 * 64));
    const int nv = static_cast<int>((width / 4 + threads - 1) / threads);
#define RUN(NV)                                                                                                        \
  hipLaunchKernelGGL(branch_norm_vec4_kernel<NV>, grid, dim3(threads), 0, stream, h, m, w1, w1_dtype, (uint16_t*)out1, \
                     w2, w2_dtype, (uint16_t*)out2, rows, width, eps)
    if (nv == 1) RUN(1);
    else if (nv == 2) RUN(2);
    else RUN(4);
#undef RUN
    return ix_check_launch("ix_branch_norm");
  }
  const dim3 block(width >= 4096 ? 1024 : (width >= 1024 ? 512 : 256));
  if (dtype == IX_F32)
    hipLaunchKernelGGL(branch_norm_kernel<float>, grid, block, 0, stream, h, m, w1, w1_dtype, (float*)out1, w2, w2_dtype,
                       (float*)out2, rows, width, eps);
  else
    hipLaunchKernelGGL(branch_norm_kernel<bf16_t>, grid, block, 0, stream, h, m, w1, w1_dtype, (bf16_t*)out1, w2, w2_dtype,
                       (bf16_t*)out2, rows, width, eps);
  return ix_check_launch("ix_branch_norm");
}
