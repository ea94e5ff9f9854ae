// Decayed linear attention over prompt portions, chunk by chunk at the same time: what
//
//     S_t = w S_(t-1) + k_t v_t^T,   o_t = S_t^T r_t          (w one number per head, S [dim, vdim] per head and request)
//
// gives for 64 rows at once is
//
//     o_i   = sum_(j <= i) w^(i - j) (r_i . k_j) v_j + w^(i + 1) S^T r_i          S: the state before the chunk
//     S_new = w^n S + sum_j w^(n - 1 - j) k_j v_j^T
//
// in three launches: every chunk's own sum of outer products (a workgroup per chunk and head), the chain over a
// request's chunks element by element (which leaves each chunk the state before it, and the request its new state),
// and every chunk's result.  All products run on the matrix cores in float32 (v_mfma_f32_32x32x2_f32), so that the
// recurrence is as exact as row by row; r, k and v come in the run's type, r and k optionally rotated (the first
// 2 * half numbers of a head, number i with i + half) and k scaled, or all three through silu, on the way into LDS.
//
// The matrix cores' operand of a 32 x 32 x 2 product is one number per lane: row (column) l % 32, reduction index
// l / 32.  Any order of the reduction indices gives the same sum, so where rows lie along the reduction (r and k in
// r . k, r and S in S^T r, the weights in their product with v) a lane reads four numbers at once: step s of eight
// takes indices 8 s + e for the lower half of the wavefront and 8 s + 4 + e for the upper, e = 0 .. 3.
#include "common.h"

typedef float f32x16 __attribute__((ext_vector_type(16)));

#define LC_ROWS 64
#define LC_COLS 128     // value columns per workgroup: a tile of 32 for each of its four wavefronts
#define LC_THREADS 256
#define LC_PS (LC_ROWS + 4)

struct LinearChunks {
  const void *r, *k, *v;          // rows of the step
  int64_t r_stride, k_stride, v_stride;
  const float* w_head;            // [heads]
  const float2* cos_sin;          // [T, half] or null
  float k_scale;
  int half, silu, heads, dim, vdim;
  const int32_t* chunk_row0;      // [chunks] first row in the step
  const int32_t* chunk_rows;      // [chunks] 1 .. 64
  float* kv;                      // [chunks, heads, vdim, dim]: a chunk's outer products, then the state before it
  float* out;                     // [T, heads, vdim]
};

__device__ __forceinline__ float lc_power(float lg, int n) { return n == 0 ? 1.0f : exp2f(static_cast<float>(n) * lg); }
__device__ __forceinline__ float lc_silu(float x) { return x / (1.0f + expf(-x)); }

// four consecutive numbers as they come from memory, opened into floats when they are used
template <typename T> struct lc_piece;
template <> struct lc_piece<float> { float4 a; };
template <> struct lc_piece<bf16_t> { uint2 a; };
__device__ __forceinline__ float4 lc_open(const lc_piece<float>& p) { return p.a; }
__device__ __forceinline__ float4 lc_open(const lc_piece<bf16_t>& p) {
  return float4{__uint_as_float(p.a.x << 16), __uint_as_float(p.a.x & 0xffff0000u), __uint_as_float(p.a.y << 16),
                __uint_as_float(p.a.y & 0xffff0000u)};
}
// four numbers of a row from d on (zeros past its `n` numbers; d < n).  VEC: the row lies on boundaries of four numbers
template <bool VEC>
__device__ __forceinline__ lc_piece<float> lc_ask(const float* row, int d, int n) {
  lc_piece<float> p;
  if constexpr (VEC) {
    p.a = *reinterpret_cast<const float4*>(row + d);
  } else {
    p.a = float4{row[d], d + 1 < n ? row[d + 1] : 0.f, d + 2 < n ? row[d + 2] : 0.f, d + 3 < n ? row[d + 3] : 0.f};
  }
  return p;
}
template <bool VEC>
__device__ __forceinline__ lc_piece<bf16_t> lc_ask(const bf16_t* row, int d, int n) {
  lc_piece<bf16_t> p;
  if constexpr (VEC) {
    p.a = *reinterpret_cast<const uint2*>(row + d);
  } else {
    const uint32_t e1 = d + 1 < n ? row[d + 1].bits : 0, e2 = d + 2 < n ? row[d + 2].bits : 0, e3 = d + 3 < n ? row[d + 3].bits : 0;
    p.a = uint2{row[d].bits | e1 << 16, e2 | e3 << 16};
  }
  return p;
}
__device__ __forceinline__ float4 lc_silu4(float4 x) { return float4{lc_silu(x.x), lc_silu(x.y), lc_silu(x.z), lc_silu(x.w)}; }
__device__ __forceinline__ float4 lc_scaled(float4 x, float f) { return float4{x.x * f, x.y * f, x.z * f, x.w * f}; }

// A tile of LC_ROWS rows of W numbers, LC_THREADS threads, four numbers each and turn: piece `u` of this thread.  Every
// piece of a tile is asked for before the first is used (rows past the chunk's last repeat it, numbers past the row's
// end repeat its first four; both are made zero on the way into LDS).
template <int W>
struct LcTile {
  static constexpr int PER = LC_ROWS * (W / 4) / LC_THREADS;
  static __device__ __forceinline__ int row(int u) { return (u * LC_THREADS + static_cast<int>(threadIdx.x)) / (W / 4); }
  static __device__ __forceinline__ int d(int u) { return 4 * ((u * LC_THREADS + static_cast<int>(threadIdx.x)) % (W / 4)); }
};

// piece u of a head's rows (of `n` numbers), and the piece it is rotated with
template <typename T, int W, bool VEC>
__device__ __forceinline__ void lc_ask_tile(const T* src, int64_t stride, int64_t row0, int rows, int n,
                                            lc_piece<T> (&p)[LcTile<W>::PER]) {
#pragma unroll
  for (int u = 0; u < LcTile<W>::PER; ++u) {
    const int d = LcTile<W>::d(u);
    p[u] = lc_ask<VEC>(src + (row0 + min(LcTile<W>::row(u), rows - 1)) * stride, d < n ? d : 0, n);
  }
}

// a piece as it enters the products: silu, or the rotation (its partners read from memory again: they are in the cache)
template <typename T, bool VEC>
__device__ __forceinline__ float4 lc_operand(const LinearChunks& a, const lc_piece<T>& p, const T* row, int64_t t, int d) {
  float4 x = lc_open(p);
  if (a.silu) return lc_silu4(x);
  if (!a.cos_sin || d >= 2 * a.half) return x;
  if (VEC && (a.half & 3) == 0) {  // four numbers of the lower half or of the upper, and four partners
    const bool low = d < a.half;
    const float4 o = lc_open(lc_ask<VEC>(row, low ? d + a.half : d - a.half, a.dim));
    const float4* cs = reinterpret_cast<const float4*>(a.cos_sin + t * a.half + (low ? d : d - a.half));
    const float4 c0 = cs[0], c1 = cs[1];  // (cos, sin) of four angles
    const float sg = low ? -1.0f : 1.0f;
    return float4{x.x * c0.x + o.x * (sg * c0.y), x.y * c0.z + o.y * (sg * c0.w), x.z * c1.x + o.z * (sg * c1.y),
                  x.w * c1.z + o.w * (sg * c1.w)};
  }
  float y[4] = {x.x, x.y, x.z, x.w};
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const int i = d + e;
    if (i >= 2 * a.half) continue;
    const bool low = i < a.half;
    const float2 c = a.cos_sin[t * a.half + (low ? i : i - a.half)];
    const float other = ix_load(row + (low ? i + a.half : i - a.half));
    y[e] = low ? y[e] * c.x - other * c.y : y[e] * c.x + other * c.y;
  }
  return float4{y[0], y[1], y[2], y[3]};
}

template <typename T, int DIM, bool VEC>
__global__ void __launch_bounds__(LC_THREADS) lc_outer_kernel(LinearChunks a) {
  __shared__ __attribute__((aligned(16))) float k_s[LC_ROWS * DIM];
  __shared__ __attribute__((aligned(16))) float v_s[LC_ROWS * LC_COLS];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int head = blockIdx.x, chunk = blockIdx.y, v0 = blockIdx.z * LC_COLS;
  const int64_t row0 = a.chunk_row0[chunk];
  const int n = a.chunk_rows[chunk];
  const float lg = log2f(a.w_head[head]);
  const T* k = static_cast<const T*>(a.k) + static_cast<int64_t>(head) * a.dim;
  const T* v = static_cast<const T*>(a.v) + static_cast<int64_t>(head) * a.vdim + v0;
  const int cols = min(LC_COLS, a.vdim - v0);
  const int n2 = (n + 1) & ~1;  // (rows are taken in pairs)
  const float4 zero = float4{0.f, 0.f, 0.f, 0.f};
  {
    lc_piece<T> kp[LcTile<DIM>::PER], vp[LcTile<LC_COLS>::PER];
    lc_ask_tile<T, DIM, VEC>(k, a.k_stride, row0, n, a.dim, kp);
    lc_ask_tile<T, LC_COLS, VEC>(v, a.v_stride, row0, n, cols, vp);
#pragma unroll
    for (int u = 0; u < LcTile<DIM>::PER; ++u) {
      const int row = LcTile<DIM>::row(u), d = LcTile<DIM>::d(u);
      float4 x = zero;
      if (row < n && d < a.dim)
        x = lc_scaled(lc_operand<T, VEC>(a, kp[u], k + (row0 + row) * a.k_stride, row0 + row, d), a.k_scale * lc_power(lg, n - 1 - row));
      *reinterpret_cast<float4*>(k_s + row * DIM + d) = x;
    }
#pragma unroll
    for (int u = 0; u < LcTile<LC_COLS>::PER; ++u) {
      const int row = LcTile<LC_COLS>::row(u), d = LcTile<LC_COLS>::d(u);
      float4 x = (row < n && d < cols) ? lc_open(vp[u]) : zero;
      if (a.silu) x = lc_silu4(x);
      *reinterpret_cast<float4*>(v_s + row * LC_COLS + d) = x;
    }
  }
  __syncthreads();
  if (32 * wave >= cols) return;
  const int c = lane & 31, h = lane >> 5;
  f32x16 acc[DIM / 32];
#pragma unroll
  for (int b = 0; b < DIM / 32; ++b)
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[b][i] = 0.f;
#pragma unroll 4
  for (int j = 0; j < n2; j += 2) {
    const float av = v_s[(j + h) * LC_COLS + 32 * wave + c];
#pragma unroll
    for (int b = 0; b < DIM / 32; ++b)
      acc[b] = __builtin_amdgcn_mfma_f32_32x32x2f32(av, k_s[(j + h) * DIM + 32 * b + c], acc[b], 0, 0, 0);
  }
  float* dst = a.kv + ((static_cast<int64_t>(chunk) * a.heads + head) * a.vdim + v0 + 32 * wave) * a.dim;
#pragma unroll
  for (int b = 0; b < DIM / 32; ++b)
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int vr = 8 * (i >> 2) + 4 * h + (i & 3), d = 32 * b + c;
      if (32 * wave + vr < cols && d < a.dim) dst[static_cast<int64_t>(vr) * a.dim + d] = acc[b][i];
    }
}

// the chain: request blockIdx.z's chunks [first, first + count) one after the other, an element (or four) per thread
template <int E>
__global__ void __launch_bounds__(256)
lc_chain_kernel(float* __restrict__ kv, const float* __restrict__ w_head, const int32_t* __restrict__ chunk_rows,
                const int32_t* __restrict__ seq_first, const int32_t* __restrict__ seq_count,
                const int32_t* __restrict__ seq_ids, const int32_t* __restrict__ state_slots, float* __restrict__ state,
                int64_t state_stride, int heads, int64_t per_head) {
  const int64_t at = (static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x) * E;
  if (at >= per_head) return;
  const int head = blockIdx.y, s = blockIdx.z;
  const float lg = log2f(w_head[head]);
  float* sp = state + static_cast<int64_t>(state_slots[seq_ids[s]]) * state_stride + head * per_head + at;
  float x[E];
#pragma unroll
  for (int e = 0; e < E; ++e) x[e] = sp[e];
  const int first = seq_first[s], count = seq_count[s];
  const int64_t step = static_cast<int64_t>(heads) * per_head;
  float* p = kv + first * step + head * per_head + at;
#pragma unroll 4
  for (int c = 0; c < count; ++c, p += step) {
    float y[E];
    if constexpr (E == 4) {
      const float4 t = *reinterpret_cast<const float4*>(p);
      y[0] = t.x; y[1] = t.y; y[2] = t.z; y[3] = t.w;
      *reinterpret_cast<float4*>(p) = float4{x[0], x[1], x[2], x[3]};
    } else {
      y[0] = *p;
      *p = x[0];
    }
    const float f = lc_power(lg, chunk_rows[first + c]);
#pragma unroll
    for (int e = 0; e < E; ++e) x[e] = f * x[e] + y[e];
  }
#pragma unroll
  for (int e = 0; e < E; ++e) sp[e] = x[e];
}

template <typename T, int DIM, bool VEC>
__global__ void __launch_bounds__(LC_THREADS) lc_result_kernel(LinearChunks a) {
  constexpr int LD = DIM + 4;  // (rows of a tile read at one place then fall on different banks)
  __shared__ __attribute__((aligned(16))) float r_s[LC_ROWS * LD];
  __shared__ __attribute__((aligned(16))) float k_s[LC_ROWS * LD];
  __shared__ __attribute__((aligned(16))) float v_s[LC_ROWS * LC_COLS];
  __shared__ __attribute__((aligned(16))) float p_s[LC_ROWS * LC_PS];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int c = lane & 31, h = lane >> 5;
  const int head = blockIdx.x, chunk = blockIdx.y, v0 = blockIdx.z * LC_COLS;
  const int64_t row0 = a.chunk_row0[chunk];
  const int n = a.chunk_rows[chunk];
  const float lg = log2f(a.w_head[head]);
  const int cols = min(LC_COLS, a.vdim - v0);
  const bool works = 32 * wave < cols;  // this wavefront has value columns
  const bool two = n > 32;              // the second tile of 32 rows holds any
  // the state before the chunk, this wavefront's columns: on its way while the rows are staged
  float4 st[DIM / 8];
  {
    const int col = v0 + 32 * wave + c;
    const float* sp = a.kv + ((static_cast<int64_t>(chunk) * a.heads + head) * a.vdim + min(col, a.vdim - 1)) * a.dim;
#pragma unroll
    for (int s = 0; s < DIM / 8; ++s) {
      const int d = 8 * s + 4 * h;
      st[s] = (works && d < a.dim) ? *reinterpret_cast<const float4*>(sp + d) : float4{0.f, 0.f, 0.f, 0.f};
    }
  }
  const T* r = static_cast<const T*>(a.r) + static_cast<int64_t>(head) * a.dim;
  const T* k = static_cast<const T*>(a.k) + static_cast<int64_t>(head) * a.dim;
  const T* v = static_cast<const T*>(a.v) + static_cast<int64_t>(head) * a.vdim + v0;
  {
    const float4 zero = float4{0.f, 0.f, 0.f, 0.f};
    lc_piece<T> rp[LcTile<DIM>::PER], kp[LcTile<DIM>::PER], vp[LcTile<LC_COLS>::PER];
    lc_ask_tile<T, DIM, VEC>(r, a.r_stride, row0, n, a.dim, rp);
    lc_ask_tile<T, DIM, VEC>(k, a.k_stride, row0, n, a.dim, kp);
    lc_ask_tile<T, LC_COLS, VEC>(v, a.v_stride, row0, n, cols, vp);
#pragma unroll
    for (int u = 0; u < LcTile<DIM>::PER; ++u) {
      const int row = LcTile<DIM>::row(u), d = LcTile<DIM>::d(u);
      float4 x = zero, y = zero;
      if (row < n && d < a.dim) {
        x = lc_operand<T, VEC>(a, rp[u], r + (row0 + row) * a.r_stride, row0 + row, d);
        y = lc_scaled(lc_operand<T, VEC>(a, kp[u], k + (row0 + row) * a.k_stride, row0 + row, d), a.k_scale);
      }
      *reinterpret_cast<float4*>(r_s + row * LD + d) = x;
      *reinterpret_cast<float4*>(k_s + row * LD + d) = y;
    }
#pragma unroll
    for (int u = 0; u < LcTile<LC_COLS>::PER; ++u) {
      const int row = LcTile<LC_COLS>::row(u), d = LcTile<LC_COLS>::d(u);
      float4 x = (row < n && d < cols) ? lc_open(vp[u]) : zero;
      if (a.silu) x = lc_silu4(x);
      *reinterpret_cast<float4*>(v_s + row * LC_COLS + d) = x;
    }
  }
  __syncthreads();
  // ---- the weights w^(i - j) (r_i . k_j), j <= i: a tile of 32 x 32 per wavefront (the one above the diagonal is empty)
  {
    const int mi = wave >> 1, ni = wave & 1;
    if (ni <= mi && (mi == 0 || two)) {
      f32x16 s;
#pragma unroll
      for (int i = 0; i < 16; ++i) s[i] = 0.f;
      const float* rp = r_s + (32 * mi + c) * LD + 4 * h;
      const float* kp = k_s + (32 * ni + c) * LD + 4 * h;
#pragma unroll 4
      for (int q = 0; q < DIM / 8; ++q) {
        const float4 x = *reinterpret_cast<const float4*>(rp + 8 * q), y = *reinterpret_cast<const float4*>(kp + 8 * q);
        s = __builtin_amdgcn_mfma_f32_32x32x2f32(x.x, y.x, s, 0, 0, 0);
        s = __builtin_amdgcn_mfma_f32_32x32x2f32(x.y, y.y, s, 0, 0, 0);
        s = __builtin_amdgcn_mfma_f32_32x32x2f32(x.z, y.z, s, 0, 0, 0);
        s = __builtin_amdgcn_mfma_f32_32x32x2f32(x.w, y.w, s, 0, 0, 0);
      }
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int ri = 32 * mi + 8 * (i >> 2) + 4 * h + (i & 3), cj = 32 * ni + c;
        p_s[ri * LC_PS + cj] = cj <= ri ? s[i] * lc_power(lg, ri - cj) : 0.f;
      }
    }
  }
  __syncthreads();
  if (!works) return;
  f32x16 o[2];
#pragma unroll
  for (int m = 0; m < 2; ++m)
#pragma unroll
    for (int i = 0; i < 16; ++i) o[m][i] = 0.f;
  // ---- S^T r
#pragma unroll
  for (int s = 0; s < DIM / 8; ++s) {
    const float4 x0 = *reinterpret_cast<const float4*>(r_s + c * LD + 8 * s + 4 * h);
    o[0] = __builtin_amdgcn_mfma_f32_32x32x2f32(x0.x, st[s].x, o[0], 0, 0, 0);
    o[0] = __builtin_amdgcn_mfma_f32_32x32x2f32(x0.y, st[s].y, o[0], 0, 0, 0);
    o[0] = __builtin_amdgcn_mfma_f32_32x32x2f32(x0.z, st[s].z, o[0], 0, 0, 0);
    o[0] = __builtin_amdgcn_mfma_f32_32x32x2f32(x0.w, st[s].w, o[0], 0, 0, 0);
    if (two) {
      const float4 x1 = *reinterpret_cast<const float4*>(r_s + (32 + c) * LD + 8 * s + 4 * h);
      o[1] = __builtin_amdgcn_mfma_f32_32x32x2f32(x1.x, st[s].x, o[1], 0, 0, 0);
      o[1] = __builtin_amdgcn_mfma_f32_32x32x2f32(x1.y, st[s].y, o[1], 0, 0, 0);
      o[1] = __builtin_amdgcn_mfma_f32_32x32x2f32(x1.z, st[s].z, o[1], 0, 0, 0);
      o[1] = __builtin_amdgcn_mfma_f32_32x32x2f32(x1.w, st[s].w, o[1], 0, 0, 0);
    }
  }
#pragma unroll
  for (int m = 0; m < 2; ++m)
#pragma unroll
    for (int i = 0; i < 16; ++i) o[m][i] *= lc_power(lg, 32 * m + 8 * (i >> 2) + 4 * h + (i & 3) + 1);
  // ---- the weights times v
#pragma unroll
  for (int s = 0; s < LC_ROWS / 8; ++s) {
    if (s >= 4 && !two) break;
    const float* vp = v_s + (8 * s + 4 * h) * LC_COLS + 32 * wave + c;
    const float b0 = vp[0], b1 = vp[LC_COLS], b2 = vp[2 * LC_COLS], b3 = vp[3 * LC_COLS];
    if (s < 4) {
      const float4 x = *reinterpret_cast<const float4*>(p_s + c * LC_PS + 8 * s + 4 * h);
      o[0] = __builtin_amdgcn_mfma_f32_32x32x2f32(x.x, b0, o[0], 0, 0, 0);
      o[0] = __builtin_amdgcn_mfma_f32_32x32x2f32(x.y, b1, o[0], 0, 0, 0);
      o[0] = __builtin_amdgcn_mfma_f32_32x32x2f32(x.z, b2, o[0], 0, 0, 0);
      o[0] = __builtin_amdgcn_mfma_f32_32x32x2f32(x.w, b3, o[0], 0, 0, 0);
    }
    if (two) {
      const float4 x = *reinterpret_cast<const float4*>(p_s + (32 + c) * LC_PS + 8 * s + 4 * h);
      o[1] = __builtin_amdgcn_mfma_f32_32x32x2f32(x.x, b0, o[1], 0, 0, 0);
      o[1] = __builtin_amdgcn_mfma_f32_32x32x2f32(x.y, b1, o[1], 0, 0, 0);
      o[1] = __builtin_amdgcn_mfma_f32_32x32x2f32(x.z, b2, o[1], 0, 0, 0);
      o[1] = __builtin_amdgcn_mfma_f32_32x32x2f32(x.w, b3, o[1], 0, 0, 0);
    }
  }
  if (32 * wave + c < cols) {
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int ri = 32 * m + 8 * (i >> 2) + 4 * h + (i & 3);
        if (ri < n) a.out[((row0 + ri) * a.heads + head) * a.vdim + v0 + 32 * wave + c] = o[m][i];
      }
  }
}

extern "C" int ix_linear_chunks(const void* r, const void* k, const void* v, int dtype, int64_t r_stride, int64_t k_stride,
                                int64_t v_stride, const float* w_head, const float* cos_sin, int half, float k_scale,
                                int silu, float* state, int64_t state_stride, const int32_t* state_slots,
                                const int32_t* chunk_row0, const int32_t* chunk_rows, int chunks,
                                const int32_t* seq_ids, const int32_t* seq_first, const int32_t* seq_count, int seqs,
                                float* kv, float* out, int heads, int dim, int vdim, hipStream_t stream) {
  IX_REQUIRE(chunks >= 0 && seqs >= 0 && heads > 0 && dim > 0 && vdim > 0, "sizes must be positive");
  IX_REQUIRE(dim <= 128 && dim % 4 == 0, "a head's keys: a multiple of four numbers, at most 128");
  IX_REQUIRE(half >= 0 && 2 * half <= dim && (half == 0 || cos_sin != nullptr), "the rotated pairs must fit into the head");
  IX_REQUIRE(half == 0 || !silu, "either a rotation or silu");
  IX_REQUIRE(state_stride >= static_cast<int64_t>(heads) * dim * vdim, "a slot's state is too small");
  IX_REQUIRE(dtype == IX_F32 || dtype == IX_BF16, "dtype must be float32 or bfloat16");
  IX_REQUIRE(heads < 65536 && chunks < 65536 && seqs < 65536, "too many heads, chunks or requests for one launch");
  IX_REQUIRE((reinterpret_cast<uintptr_t>(kv) & 15) == 0, "the workspace must lie on a 16-byte boundary");
  if (chunks == 0 || seqs == 0) return 0;
  LinearChunks a;
  a.r = r; a.k = k; a.v = v; a.r_stride = r_stride; a.k_stride = k_stride; a.v_stride = v_stride;
  a.w_head = w_head; a.cos_sin = half > 0 ? reinterpret_cast<const float2*>(cos_sin) : nullptr; a.k_scale = k_scale;
  a.half = half; a.silu = silu; a.heads = heads; a.dim = dim; a.vdim = vdim;
  a.chunk_row0 = chunk_row0; a.chunk_rows = chunk_rows; a.kv = kv; a.out = out;
  const uintptr_t rows = reinterpret_cast<uintptr_t>(r) | reinterpret_cast<uintptr_t>(k) | reinterpret_cast<uintptr_t>(v);
  const bool vec = (rows & 15) == 0 && (r_stride | k_stride | v_stride) % 4 == 0 && vdim % 4 == 0;
  dim3 grid(heads, chunks, (vdim + LC_COLS - 1) / LC_COLS), block(LC_THREADS);
  const int64_t per_head = static_cast<int64_t>(dim) * vdim;
  const bool fours = per_head % 4 == 0 && state_stride % 4 == 0 && (reinterpret_cast<uintptr_t>(state) & 15) == 0;
  const int64_t threads = fours ? per_head / 4 : per_head;
  dim3 chain(static_cast<unsigned>((threads + 255) / 256), heads, seqs);
#define BY_DIM(KERNEL, T, VEC)                                                                       \
  if (dim <= 32) hipLaunchKernelGGL((KERNEL<T, 32, VEC>), grid, block, 0, stream, a);                \
  else if (dim <= 64) hipLaunchKernelGGL((KERNEL<T, 64, VEC>), grid, block, 0, stream, a);           \
  else if (dim <= 96) hipLaunchKernelGGL((KERNEL<T, 96, VEC>), grid, block, 0, stream, a);           \
  else hipLaunchKernelGGL((KERNEL<T, 128, VEC>), grid, block, 0, stream, a)
#define BY_TYPE(KERNEL)                                     \
  if (dtype == IX_F32 && vec) { BY_DIM(KERNEL, float, true); }   \
  else if (dtype == IX_F32) { BY_DIM(KERNEL, float, false); }    \
  else if (vec) { BY_DIM(KERNEL, bf16_t, true); }                \
  else { BY_DIM(KERNEL, bf16_t, false); }
  BY_TYPE(lc_outer_kernel)
  if (ix_check_launch("ix_linear_chunks: outer products")) return 1;
  if (fours)
    hipLaunchKernelGGL(lc_chain_kernel<4>, chain, dim3(256), 0, stream, kv, w_head, chunk_rows, seq_first, seq_count, seq_ids,
                       state_slots, state, state_stride, heads, per_head);
  else
    hipLaunchKernelGGL(lc_chain_kernel<1>, chain, dim3(256), 0, stream, kv, w_head, chunk_rows, seq_first, seq_count, seq_ids,
                       state_slots, state, state_stride, heads, per_head);
  if (ix_check_launch("ix_linear_chunks: chain")) return 1;
  BY_TYPE(lc_result_kernel)
#undef BY_TYPE
#undef BY_DIM
  return ix_check_launch("ix_linear_chunks");
}
