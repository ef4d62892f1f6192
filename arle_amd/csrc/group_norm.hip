// RMS norm in groups over rows, with the adds of a parallel block fused in.
//
//   x_j   = src_j + t0_j + t1_j + t2_j                                  (32-bit; written back to the residual)
//   out_j = x_j / sqrt(mean of x^2 over the group of j + eps) * w_j
//
// A row of `width` entries is `groups` equal groups of consecutive entries; with one group it is the plain RMS norm.
// `plain`: no norm and no weight, out_j = x_j (the sum of the residual and the terms in another type).  The terms are what the sublayers in front left to be added (addend.h: tensors, stacks of partial sums, weighted
// outputs of experts, a factor per row).  The source is the float32 residual, or rows of a table picked by index (an
// embedding that is normed on its way into the residual); rows picked by index are not written back.  Statistics, sums
// and the weight are 32-bit; a row's arithmetic depends on nothing but the row.
#include "addend.h"

namespace arle {

struct Terms {
  Addend t[3];
};

// A group's sum of squares is made of one partial sum an access of four entries, laid down in LDS and added by one wave
// in an order that depends on the group's size alone.
template <int THREADS>
__device__ __forceinline__ void group_scales(const float* ssq, float* inv, int groups, int pieces, float size, float eps) {
  const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
  for (int g = wave; g < groups; g += THREADS / kWave) {
    float s = 0.f;
    for (int i = lane; i < pieces; i += kWave) s += ssq[g * pieces + i];
    s = wave_sum(s);
    if (lane == 0) inv[g] = 1.0f / sqrtf(s / size + eps);
  }
}

// Four entries a thread and access (group sizes that are multiples of 4, 16-byte aligned rows), the row in registers.
template <typename TIn, typename TOut, typename TW, int THREADS, int VPT>
__global__ __launch_bounds__(THREADS) void group_norm_vec_kernel(const TIn* __restrict__ x, int64_t x_stride,
                                                                 float* __restrict__ back, const Terms terms,
                                                                 const TW* __restrict__ w, TOut* __restrict__ out, int64_t out_stride,
                                                                 const int* __restrict__ rows, int width, int groups,
                                                                 float eps, int plain) {
  extern __shared__ float lds[];   // [width / 4] partial sums of squares, then [groups] scales
  float* ssq = lds;
  float* inv = lds + width / 4;
  const int64_t r = blockIdx.x, src = rows ? rows[r] : r;
  const int tid = threadIdx.x, last = width - 4;
  float4 v[VPT], wv[VPT];
  int at[VPT];
  // no load stands under a condition: a piece past the width is the last one again, left out of sums and stores
#pragma unroll
  for (int j = 0; j < VPT; ++j) {
    at[j] = min(4 * (tid + j * THREADS), last);
    v[j] = ld4<TIn>(x + src * x_stride + at[j]);
    wv[j] = ld4<TW>(w + at[j]);
  }
#pragma unroll
  for (int k = 0; k < 3; ++k) {
    const Addend& a = terms.t[k];
    if (!a.p) continue;
    const float* base = a.p + src * a.row_stride;
    float4 sum[VPT];
#pragma unroll
    for (int j = 0; j < VPT; ++j) sum[j] = float4{0.f, 0.f, 0.f, 0.f};
    constexpr int G = VPT <= 2 ? 4 : 2;     // parts in flight at a time
    for (int p0 = 0; p0 < a.parts; p0 += G) {
      float4 e[G][VPT];
      float f[G];
#pragma unroll
      for (int u = 0; u < G; ++u) {
        const int p = min(p0 + u, a.parts - 1);
#pragma unroll
        for (int j = 0; j < VPT; ++j) e[u][j] = ld4<float>(base + p * a.part_stride + at[j]);
        f[u] = a.weights ? a.weights[src * a.w_row + p * a.w_part] : 1.0f;
      }
#pragma unroll
      for (int u = 0; u < G; ++u) {
        const bool in = p0 + u < a.parts;
        const float fu = in ? f[u] : 0.f;
#pragma unroll
        for (int j = 0; j < VPT; ++j) {
          if (in) {
            sum[j].x = fmaf(fu, e[u][j].x, sum[j].x); sum[j].y = fmaf(fu, e[u][j].y, sum[j].y);
            sum[j].z = fmaf(fu, e[u][j].z, sum[j].z); sum[j].w = fmaf(fu, e[u][j].w, sum[j].w);
          }
        }
      }
    }
#pragma unroll
    for (int j = 0; j < VPT; ++j) {
      v[j].x += sum[j].x; v[j].y += sum[j].y; v[j].z += sum[j].z; v[j].w += sum[j].w;
    }
  }
#pragma unroll
  for (int j = 0; j < VPT; ++j) {
    const int i = 4 * (tid + j * THREADS);
    if (i < width) {
      if (back) st4<float>(back + src * width + i, v[j]);
      ssq[i / 4] = (v[j].x * v[j].x + v[j].y * v[j].y) + (v[j].z * v[j].z + v[j].w * v[j].w);
    }
  }
  if (plain) {
#pragma unroll
    for (int j = 0; j < VPT; ++j) {
      const int i = 4 * (tid + j * THREADS);
      if (i < width) st4<TOut>(out + r * out_stride + i, v[j]);
    }
    return;
  }
  __syncthreads();
  const int size = width / groups;
  group_scales<THREADS>(ssq, inv, groups, size / 4, static_cast<float>(size), eps);
  __syncthreads();
#pragma unroll
  for (int j = 0; j < VPT; ++j) {
    const int i = 4 * (tid + j * THREADS);
    if (i < width) {
      const float s = inv[i / size];
      st4<TOut>(out + r * out_stride + i, float4{v[j].x * s * wv[j].x, v[j].y * s * wv[j].y, v[j].z * s * wv[j].z, v[j].w * s * wv[j].w});
    }
  }
}

constexpr int kGroupThreads = 256;

// Any sizes and alignment: one entry a thread and access, the row in LDS.
template <typename TIn, typename TOut, typename TW>
__global__ __launch_bounds__(kGroupThreads) void group_norm_kernel(const TIn* __restrict__ x, int64_t x_stride,
                                                                   float* __restrict__ back, const Terms terms,
                                                                   const TW* __restrict__ w, TOut* __restrict__ out, int64_t out_stride,
                                                                   const int* __restrict__ rows, int width, int groups,
                                                                   float eps, int plain) {
  extern __shared__ float lds[];   // [width] the row, then [groups] scales
  float* xs = lds;
  float* inv = lds + width;
  const int64_t r = blockIdx.x, src = rows ? rows[r] : r;
  for (int i = threadIdx.x; i < width; i += kGroupThreads) {
    float v = to_float(x[src * x_stride + i]);
#pragma unroll
    for (int k = 0; k < 3; ++k) {
      const Addend& a = terms.t[k];
      if (!a.p) continue;
      const float* base = a.p + src * a.row_stride + i;
      float sum = 0.f;
      for (int p = 0; p < a.parts; ++p)
        sum = fmaf(a.weights ? a.weights[src * a.w_row + p * a.w_part] : 1.0f, base[p * a.part_stride], sum);
      v += sum;
    }
    if (back) back[src * width + i] = v;
    if (plain) out[r * out_stride + i] = from_float<TOut>(v);
    xs[i] = v;
  }
  if (plain) return;
  __syncthreads();
  const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave, size = width / groups;
  for (int g = wave; g < groups; g += kGroupThreads / kWave) {
    float s = 0.f;
    for (int i = lane; i < size; i += kWave) s = fmaf(xs[g * size + i], xs[g * size + i], s);
    s = wave_sum(s);
    if (lane == 0) inv[g] = 1.0f / sqrtf(s / static_cast<float>(size) + eps);
  }
  __syncthreads();
  for (int i = threadIdx.x; i < width; i += kGroupThreads)
    out[r * out_stride + i] = from_float<TOut>(xs[i] * inv[i / size] * to_float(w[i]));
}

constexpr int kGroupLdsMax = 128 * 1024;   // [width] + [groups] floats of the plain kernel at width 16384, one group an entry

template <typename TIn, typename TOut, typename TW>
static int launch_group_norm(const void* x, long long x_stride, float* back, const Terms& terms, const void* w, void* out,
                             long long out_stride, const int* rows, int n_rows, int width, int groups, float eps, int plain,
                             bool vec, hipStream_t s) {
  const TIn* xp = static_cast<const TIn*>(x);
  const TW* wp = static_cast<const TW*>(w);
  TOut* op = static_cast<TOut*>(out);
  if (vec) {
    const size_t lds = static_cast<size_t>(width / 4 + groups) * sizeof(float);   // at most 32 KB
#define ARLE_GN(THREADS, VPT)                                                                                          \
  group_norm_vec_kernel<TIn, TOut, TW, THREADS, VPT><<<n_rows, THREADS, lds, s>>>(xp, x_stride, back, terms, wp, op, \
                                                                                  out_stride, rows, width, groups, eps, plain)
    if (width <= 1024) {
      ARLE_GN(256, 1);
    } else if (n_rows <= 512 && width <= 4096) {   // few rows: the latency of one access a thread
      ARLE_GN(1024, 1);
    } else if (width <= 2048) {
      ARLE_GN(256, 2);
    } else if (width <= 4096) {
      ARLE_GN(256, 4);
    } else if (width <= 8192) {
      ARLE_GN(1024, 2);
    } else {
      ARLE_GN(1024, 4);
    }
#undef ARLE_GN
    return launch_status();
  }
  const size_t lds = static_cast<size_t>(width + groups) * sizeof(float);
  static bool raised = false;
  if (!raised && lds > 48 * 1024) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&group_norm_kernel<TIn, TOut, TW>),
                                             hipFuncAttributeMaxDynamicSharedMemorySize, kGroupLdsMax);
    if (e != hipSuccess) return static_cast<int>(e);
    raised = true;
  }
  group_norm_kernel<TIn, TOut, TW><<<n_rows, kGroupThreads, lds, s>>>(xp, x_stride, back, terms, wp, op, out_stride, rows,
                                                                      width, groups, eps, plain);
  return launch_status();
}

}  // namespace arle

using namespace arle;

// x: rows of x_dtype, x_stride elements apart; back: float32 [*, width] that the sums are written to (the residual, which
// x then is), or null.  Three addends (null pointers: none), float32, indexed like x.  out [n_rows, width] of out_dtype,
// rows out_stride apart; plain: see above (w then is any `width` readable entries of w_dtype).
// rows: which rows of x (null: 0..n_rows-1).  groups divides width; width <= 16384.
extern "C" int arle_group_norm(const void* x, int x_dtype, long long x_stride, float* back, const float* a, int a_parts,
                               long long a_part_stride, long long a_row_stride, const float* a_weights, int a_w_row,
                               int a_w_part, const float* b, int b_parts, long long b_part_stride, long long b_row_stride,
                               const float* b_weights, int b_w_row, int b_w_part, const float* c, int c_parts,
                               long long c_part_stride, long long c_row_stride, const float* c_weights, int c_w_row,
                               int c_w_part, const void* w, int w_dtype, void* out, long long out_stride,
                               int out_dtype, const int* rows, int n_rows, int width, int groups, float eps, int plain,
                               void* stream) {
  if (n_rows == 0) return 0;
  if (width < 1 || width > 16384 || groups < 1 || width % groups || (a && a_parts < 1) || (b && b_parts < 1) || (c && c_parts < 1))
    return static_cast<int>(hipErrorInvalidValue);
  const Terms terms{{{a, a_parts, a_part_stride, a_row_stride, a_weights, a_w_row, a_w_part},
                     {b, b_parts, b_part_stride, b_row_stride, b_weights, b_w_row, b_w_part},
                     {c, c_parts, c_part_stride, c_row_stride, c_weights, c_w_row, c_w_part}}};
  auto al = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  bool vec = (width / groups) % 4 == 0 && x_stride % 4 == 0 && al(x) && al(back) && al(w) && al(out) && out_stride % 4 == 0;
  for (const Addend& t : terms.t) vec = vec && (!t.p || (al(t.p) && t.part_stride % 4 == 0 && t.row_stride % 4 == 0));
  hipStream_t s = static_cast<hipStream_t>(stream);
#define ARLE_GNL(TI, TO, TWT) \
  return launch_group_norm<TI, TO, TWT>(x, x_stride, back, terms, w, out, out_stride, rows, n_rows, width, groups, eps, plain, vec, s)
#define ARLE_GNO(TI, TO)                                          \
  do {                                                            \
    if (w_dtype == kF32) ARLE_GNL(TI, TO, float);                 \
    ARLE_GNL(TI, TO, bf16);                                       \
  } while (0)
  if (x_dtype == kF32) {
    if (out_dtype == kF32) ARLE_GNO(float, float);
    ARLE_GNO(float, bf16);
  }
  if (out_dtype == kF32) ARLE_GNO(bf16, float);
  ARLE_GNO(bf16, bf16);
#undef ARLE_GNO
#undef ARLE_GNL
}
