// A residual stream that is kept in several copies (hyper-connections), float32 [T, S, W], and the step from one
// sublayer to the next in one pass:
//
//     x_j <- sum_i mix[i, j] x_i + gain[j] * y      the sublayer's result y comes back, all copies at once from the old
//     u    = sum_j enter[j] x_j                      what the next sublayer reads (enter null: the plain sum)
//     out  = u / sqrt(mean(u^2) + eps) * weight      its norm
//
// Without y the copies stay as they are.  With `rows` only those rows are formed (row rows[r] gives out[r]) and the
// copies are not written: the end of the model, where nobody reads them any more.
// ix_embed_norm makes the stream's start: a row of the table through an RMS norm, written S times.
// Everything is float32; y and out have the run's type.
#include "common.h"

#define STREAMS_MAX 32

__device__ __forceinline__ float4 st_load4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 st_load4(const bf16_t* p) {
  const uint2 d = *reinterpret_cast<const uint2*>(p);
  return float4{__uint_as_float(d.x << 16), __uint_as_float(d.x & 0xffff0000u), __uint_as_float(d.y << 16),
                __uint_as_float(d.y & 0xffff0000u)};
}
__device__ __forceinline__ void st_store4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
__device__ __forceinline__ void st_store4(bf16_t* p, float4 v) {
  uint2 o;
  o.x = ix_f32_to_bf16(v.x) | static_cast<uint32_t>(ix_f32_to_bf16(v.y)) << 16;
  o.y = ix_f32_to_bf16(v.z) | static_cast<uint32_t>(ix_f32_to_bf16(v.w)) << 16;
  *reinterpret_cast<uint2*>(p) = o;
}

// S copies in registers, four columns per thread and turn, PER turns (4 * PER * blockDim.x >= width)
template <int S, typename T, int PER>
__global__ void __launch_bounds__(1024)
stream_norm_vec4_kernel(float* __restrict__ h, const T* __restrict__ y, const float* __restrict__ mix,
                        const float* __restrict__ gain, const float* __restrict__ enter,
                        const float* __restrict__ weight, T* __restrict__ out, const int32_t* __restrict__ rows,
                        int width, float eps) {
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  const int64_t row = rows ? rows[r] : r;
  float* hr = h + row * S * width;
  float4 u[PER];
  float sumsq = 0.f;
#pragma unroll
  for (int p = 0; p < PER; ++p) {
    const int c = 4 * (p * blockDim.x + threadIdx.x);
    u[p] = float4{0.f, 0.f, 0.f, 0.f};
    if (c >= width) continue;
    float4 x[S];
#pragma unroll
    for (int i = 0; i < S; ++i) x[i] = st_load4(hr + static_cast<int64_t>(i) * width + c);
    if (y) {
      const float4 d = st_load4(y + row * width + c);
      float4 z[S];
#pragma unroll
      for (int j = 0; j < S; ++j) {
        const float g = gain[j];
        z[j] = float4{g * d.x, g * d.y, g * d.z, g * d.w};
#pragma unroll
        for (int i = 0; i < S; ++i) {
          const float m = mix[i * S + j];
          z[j].x += m * x[i].x;
          z[j].y += m * x[i].y;
          z[j].z += m * x[i].z;
          z[j].w += m * x[i].w;
        }
      }
#pragma unroll
      for (int j = 0; j < S; ++j) {
        x[j] = z[j];
        if (!rows) st_store4(hr + static_cast<int64_t>(j) * width + c, z[j]);
      }
    }
#pragma unroll
    for (int j = 0; j < S; ++j) {
      const float a = enter ? enter[j] : 1.0f;
      u[p].x += a * x[j].x;
      u[p].y += a * x[j].y;
      u[p].z += a * x[j].z;
      u[p].w += a * x[j].w;
    }
    sumsq += u[p].x * u[p].x + u[p].y * u[p].y + u[p].z * u[p].z + u[p].w * u[p].w;
  }
  sumsq = ix_block_sum(sumsq, red);
  const float inv = 1.0f / sqrtf(sumsq / static_cast<float>(width) + eps);
#pragma unroll
  for (int p = 0; p < PER; ++p) {
    const int c = 4 * (p * blockDim.x + threadIdx.x);
    if (c >= width) continue;
    const float4 w = st_load4(weight + c);
    st_store4(out + r * width + c, float4{u[p].x * inv * w.x, u[p].y * inv * w.y, u[p].z * inv * w.z, u[p].w * inv * w.w});
  }
}

// any width, any number of copies up to STREAMS_MAX: a column per thread and turn, the entered sum kept in `work`
// (float32 [n_out, width]) between the two passes
template <typename T>
__global__ void __launch_bounds__(256)
stream_norm_kernel(float* __restrict__ h, const T* __restrict__ y, const float* __restrict__ mix,
                   const float* __restrict__ gain, const float* __restrict__ enter, const float* __restrict__ weight,
                   T* __restrict__ out, const int32_t* __restrict__ rows, float* __restrict__ work, int streams, int width,
                   float eps) {
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  const int64_t row = rows ? rows[r] : r;
  float* hr = h + row * streams * width;
  float sumsq = 0.f;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    float x[STREAMS_MAX];
    for (int i = 0; i < streams; ++i) x[i] = hr[static_cast<int64_t>(i) * width + c];
    float u = 0.f;
    if (y) {
      const float d = ix_load(y + row * width + c);
      for (int j = 0; j < streams; ++j) {
        float z = gain[j] * d;
        for (int i = 0; i < streams; ++i) z += mix[i * streams + j] * x[i];
        if (!rows) hr[static_cast<int64_t>(j) * width + c] = z;
        u += (enter ? enter[j] : 1.0f) * z;
      }
    } else {
      for (int j = 0; j < streams; ++j) u += (enter ? enter[j] : 1.0f) * x[j];
    }
    work[r * width + c] = u;
    sumsq += u * u;
  }
  sumsq = ix_block_sum(sumsq, red);
  const float inv = 1.0f / sqrtf(sumsq / static_cast<float>(width) + eps);
  for (int c = threadIdx.x; c < width; c += blockDim.x)  // (a thread reads what it wrote itself)
    ix_store(out + r * width + c, work[r * width + c] * inv * weight[c]);
}

// whether the form without `work` takes these sizes
extern "C" int ix_stream_norm_needs_work(int streams, int64_t width) {
  return (streams <= 8 && width % 4 == 0 && width <= 16384) ? 0 : 1;
}

extern "C" int ix_stream_norm(float* h, const void* y, const float* mix, const float* gain, const float* enter,
                              const float* weight, void* out, int dtype, const int32_t* rows, float* work, int64_t n_out,
                              int streams, int64_t width, float eps, hipStream_t stream) {
  IX_REQUIRE(n_out >= 0 && streams > 0 && streams <= STREAMS_MAX && width > 0 && width < (1 << 24), "between 1 and 32 streams");
  IX_REQUIRE(dtype == IX_F32 || dtype == IX_BF16, "dtype must be float32 or bfloat16");
  IX_REQUIRE(y == nullptr || (mix != nullptr && gain != nullptr), "a result that comes back needs the mix and its gains");
  IX_REQUIRE(n_out < (1ll << 31), "too many rows for one launch");
  if (n_out == 0) return 0;
  const uintptr_t all = reinterpret_cast<uintptr_t>(h) | reinterpret_cast<uintptr_t>(y) | reinterpret_cast<uintptr_t>(weight) |
                        reinterpret_cast<uintptr_t>(out);
  dim3 grid(static_cast<unsigned>(n_out));
  const int w32 = static_cast<int>(width);
  if (!ix_stream_norm_needs_work(streams, width) && (all & 15) == 0) {
    const int quads = w32 / 4;
    int threads = 64;
    while (threads < 1024 && threads < quads) threads *= 2;
    const int per = (quads + threads - 1) / threads;
#define LAUNCH(S, T, PER)                                                                                              \
  hipLaunchKernelGGL((stream_norm_vec4_kernel<S, T, PER>), grid, dim3(threads), 0, stream, h, (const T*)y, mix, gain, enter, \
                     weight, (T*)out, rows, w32, eps)
#define BY_PER(S, T)                        \
  if (per == 1) LAUNCH(S, T, 1);            \
  else if (per == 2) LAUNCH(S, T, 2);       \
  else LAUNCH(S, T, 4)
#define CASE(S)                                       \
  case S:                                             \
    if (dtype == IX_BF16) { BY_PER(S, bf16_t); }      \
    else { BY_PER(S, float); }                        \
    break;
    switch (streams) { CASE(1) CASE(2) CASE(3) CASE(4) CASE(5) CASE(6) CASE(7) CASE(8) }
#undef CASE
#undef BY_PER
#undef LAUNCH
    return ix_check_launch("ix_stream_norm");
  }
  IX_REQUIRE(work != nullptr, "these sizes need a workspace of a float per row and column");
  if (dtype == IX_BF16)
    hipLaunchKernelGGL(stream_norm_kernel<bf16_t>, grid, dim3(256), 0, stream, h, (const bf16_t*)y, mix, gain, enter, weight,
                       (bf16_t*)out, rows, work, streams, w32, eps);
  else
    hipLaunchKernelGGL(stream_norm_kernel<float>, grid, dim3(256), 0, stream, h, (const float*)y, mix, gain, enter, weight,
                       (float*)out, rows, work, streams, w32, eps);
  return ix_check_launch("ix_stream_norm");
}

// h[t, j, :] = norm(table[ids[t], :] * scale) for every copy j; without a weight the row as it is
template <typename TW>
__global__ void __launch_bounds__(256)
embed_norm_kernel(float* __restrict__ h, const TW* __restrict__ table, const int32_t* __restrict__ ids,
                  const float* __restrict__ weight, int64_t width, int64_t vocab, int streams, float scale, float eps) {
  __shared__ float red[16];
  const int64_t t = blockIdx.x;
  const int64_t id = ids[t];
  const bool ok = id >= 0 && id < vocab;
  const TW* row = table + (ok ? id : 0) * width;
  float inv = ok ? scale : 0.f;
  if (weight) {
    float ss = 0.f;
    for (int64_t i = threadIdx.x; i < width; i += blockDim.x) {
      const float v = ix_load(row + i) * scale;
      ss += v * v;
    }
    ss = ix_block_sum(ss, red);
    inv = ok ? scale / sqrtf(ss / static_cast<float>(width) + eps) : 0.f;
  }
  for (int64_t i = threadIdx.x; i < width; i += blockDim.x) {
    float v = ix_load(row + i) * inv;
    if (weight) v *= weight[i];
    for (int j = 0; j < streams; ++j) h[(t * streams + j) * width + i] = v;
  }
}

// the same with the row in registers, four columns per thread and turn
template <typename TW, int PER>
__global__ void __launch_bounds__(1024)
embed_norm_vec4_kernel(float* __restrict__ h, const TW* __restrict__ table, const int32_t* __restrict__ ids,
                       const float* __restrict__ weight, int width, int64_t vocab, int streams, float scale, float eps) {
  __shared__ float red[16];
  const int64_t t = blockIdx.x;
  const int64_t id = ids[t];
  const bool ok = id >= 0 && id < vocab;
  const TW* row = table + (ok ? id : 0) * width;
  float4 x[PER];
  float ss = 0.f;
#pragma unroll
  for (int p = 0; p < PER; ++p) {
    const int c = 4 * (p * blockDim.x + threadIdx.x);
    x[p] = c < width ? st_load4(row + c) : float4{0.f, 0.f, 0.f, 0.f};
    x[p] = float4{x[p].x * scale, x[p].y * scale, x[p].z * scale, x[p].w * scale};
    ss += x[p].x * x[p].x + x[p].y * x[p].y + x[p].z * x[p].z + x[p].w * x[p].w;
  }
  float inv = ok ? 1.0f : 0.f;
  if (weight) {
    ss = ix_block_sum(ss, red);
    inv = ok ? 1.0f / sqrtf(ss / static_cast<float>(width) + eps) : 0.f;
  }
#pragma unroll
  for (int p = 0; p < PER; ++p) {
    const int c = 4 * (p * blockDim.x + threadIdx.x);
    if (c >= width) continue;
    const float4 w = weight ? st_load4(weight + c) : float4{1.f, 1.f, 1.f, 1.f};
    const float4 v = float4{x[p].x * inv * w.x, x[p].y * inv * w.y, x[p].z * inv * w.z, x[p].w * inv * w.w};
    for (int j = 0; j < streams; ++j) st_store4(h + (t * streams + j) * width + c, v);
  }
}

extern "C" int ix_embed_norm(float* h, const void* table, int table_dtype, const int32_t* ids, const float* weight,
                             int64_t tokens, int64_t width, int64_t vocab, int streams, float scale, float eps,
                             hipStream_t stream) {
  IX_REQUIRE(tokens >= 0 && width > 0 && vocab > 0 && streams > 0, "sizes must be positive");
  IX_REQUIRE(table_dtype == IX_F32 || table_dtype == IX_BF16, "table dtype must be float32 or bfloat16");
  IX_REQUIRE(tokens < (1ll << 31), "too many tokens for one launch");
  if (tokens == 0) return 0;
  dim3 grid(static_cast<unsigned>(tokens)), block(256);
  const uintptr_t all = reinterpret_cast<uintptr_t>(h) | reinterpret_cast<uintptr_t>(table) | reinterpret_cast<uintptr_t>(weight);
  if (width % 4 == 0 && width <= 16384 && (all & 15) == 0) {
    const int quads = static_cast<int>(width / 4);
    int threads = 64;
    while (threads < 1024 && threads < quads) threads *= 2;
    const int per = (quads + threads - 1) / threads;
#define LAUNCH(T, PER)                                                                                                  \
  hipLaunchKernelGGL((embed_norm_vec4_kernel<T, PER>), grid, dim3(threads), 0, stream, h, (const T*)table, ids, weight, \
                     static_cast<int>(width), vocab, streams, scale, eps)
#define BY_PER(T)                  \
  if (per == 1) LAUNCH(T, 1);      \
  else if (per == 2) LAUNCH(T, 2); \
  else LAUNCH(T, 4)
    if (table_dtype == IX_F32) { BY_PER(float); } else { BY_PER(bf16_t); }
#undef BY_PER
#undef LAUNCH
    return ix_check_launch("ix_embed_norm");
  }
  if (table_dtype == IX_F32)
    hipLaunchKernelGGL(embed_norm_kernel<float>, grid, block, 0, stream, h, (const float*)table, ids, weight, width, vocab,
                       streams, scale, eps);
  else
    hipLaunchKernelGGL(embed_norm_kernel<bf16_t>, grid, block, 0, stream, h, (const bf16_t*)table, ids, weight, width, vocab,
                       streams, scale, eps);
  return ix_check_launch("ix_embed_norm");
}
