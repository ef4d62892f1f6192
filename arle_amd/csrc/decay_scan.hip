// Linear attention whose state decays by numbers made from the tokens, row by row, for the rows of a packed step, continued
// across steps through a per-request state S [heads, D, Dv] in 32-bit floats.  Every sum in one order whatever a step
// holds; all arithmetic is 32-bit.
//
//   S_t = diag(decay_t) S_(t-1) + k_t v_t^T,    o_t = S_t^T q_t            (per head; head h reads q/k head h / (H / G))
//
// One decay a head (the state-space form): with dt = softplus(raw + dt_bias_h), the decay is exp(-exp(A_log_h) dt), v counts
// dt times, and D_h v_t (v without dt) is added to the read-out.
// A decay for every head and key entry (CHANNEL): a float32 tensor [T, H * D], made by `decay_gates` from the narrow middle m
// of two projections, sigmoid(z)^(1/tau) with z = W m + b: the decays themselves, or, for the form over chunks, the running
// sum of their logarithms from the chunk's first row on.  q counts D^(-1/2) times.
#include "chunks.h"
#include "lane_sums.h"

namespace arle {

constexpr int kDsThreads = 256;
constexpr int kDsCols = 16;                        // columns of S a workgroup looks after, four a wave
constexpr int kDsParts = 16;                       // shares of D, one a lane of a row of sixteen
constexpr int kDsRows = 32;                        // rows staged at a time
constexpr int kDsRowThreads = kDsThreads / kDsRows;

struct ScanArgs {
  const void* q; long long q_stride;
  const void* k; long long k_stride;
  const void* v; long long v_stride;
  const float* decay; long long decay_stride;      // CHANNEL: [T, H * D] decays; else [T, H] raw step sizes
  const float* a_log; const float* dt_bias; const float* skip;
  float q_scale;
  float* s_state;
  const int* seg_row0; const int* seg_slot;
  float* out;                                      // [T, H * Dv]
  int H, G, D, Dv;
};

template <typename T, int DS, bool CHANNEL>
__global__ __launch_bounds__(kDsThreads) void decay_scan_kernel(const ScanArgs a) {
  constexpr int DP = kDsParts * DS;                // padded D: what lies past D is zero
  constexpr int kMine = DP / kDsRowThreads, kValues = kDsRows * kDsCols / kDsThreads;
  __shared__ float q_lds[kDsRows][DP], k_lds[kDsRows][DP];
  __shared__ float g_lds[CHANNEL ? kDsRows : 1][DP];
  __shared__ float v_lds[kDsRows][kDsCols];
  __shared__ float c_lds[kDsRows][2];              // !CHANNEL: decay, dt
  const int seg = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave;
  const int kvh = h / (a.H / a.G), D = a.D, Dv = a.Dv;
  const int col_in = wave * 4 + lane / kDsParts, col = blockIdx.z * kDsCols + col_in, part = lane % kDsParts;
  const bool live = col < Dv;
  const int row0 = a.seg_row0[seg], rows = a.seg_row0[seg + 1] - row0;
  float* s_ptr = a.s_state + (static_cast<int64_t>(a.seg_slot[seg]) * a.H + h) * D * Dv;
  const T* q = static_cast<const T*>(a.q);
  const T* k = static_cast<const T*>(a.k);
  const T* v = static_cast<const T*>(a.v);
  const float rate = CHANNEL ? 0.f : expf(a.a_log[h]), bias = CHANNEL ? 0.f : a.dt_bias[h], skip = CHANNEL ? 0.f : a.skip[h];
  float S[DS];
#pragma unroll
  for (int i = 0; i < DS; ++i) {
    const int d = part * DS + i;
    S[i] = (live && d < D) ? s_ptr[static_cast<int64_t>(d) * Dv + col] : 0.f;
  }
  const int r = tid / kDsRowThreads, sub = tid % kDsRowThreads;
  float q_next[kMine], k_next[kMine], g_next[CHANNEL ? kMine : 1], v_next[kValues], c_next = 0.f;
  auto fetch = [&](int base) {
    const int n = min(kDsRows, rows - base);       // <= 0 behind the last block: nothing is loaded
    const int64_t t = row0 + base + min(r, max(n, 1) - 1);
#pragma unroll
    for (int j = 0; j < kMine; ++j) {
      const int d = sub + j * kDsRowThreads;
      const bool there = r < n && d < D;
      q_next[j] = there ? to_float(q[t * a.q_stride + kvh * D + d]) : 0.f;
      k_next[j] = there ? to_float(k[t * a.k_stride + kvh * D + d]) : 0.f;
      if constexpr (CHANNEL) g_next[j] = there ? a.decay[t * a.decay_stride + h * D + d] : 0.f;
    }
    if constexpr (!CHANNEL) c_next = (sub == 0 && r < n) ? a.decay[t * a.decay_stride + h] : 0.f;
#pragma unroll
    for (int j = 0; j < kValues; ++j) {
      const int e = tid + j * kDsThreads, rr = e / kDsCols, c = blockIdx.z * kDsCols + e % kDsCols;
      v_next[j] = (rr < n && c < Dv) ? to_float(v[(row0 + base + rr) * a.v_stride + h * Dv + c]) : 0.f;
    }
  };
  fetch(0);
  for (int base = 0; base < rows; base += kDsRows) {
    const int n = min(kDsRows, rows - base);
    __syncthreads();                               // the block before has been read
#pragma unroll
    for (int j = 0; j < kMine; ++j) {
      q_lds[r][sub + j * kDsRowThreads] = q_next[j] * a.q_scale;
      k_lds[r][sub + j * kDsRowThreads] = k_next[j];
      if constexpr (CHANNEL) g_lds[r][sub + j * kDsRowThreads] = g_next[j];
    }
    if constexpr (!CHANNEL) {
      if (sub == 0) {
        const float dt = softplus_f(c_next + bias);
        c_lds[r][0] = expf(-rate * dt);
        c_lds[r][1] = dt;
      }
    }
#pragma unroll
    for (int j = 0; j < kValues; ++j) v_lds[(tid + j * kDsThreads) / kDsCols][(tid + j * kDsThreads) % kDsCols] = v_next[j];
    __syncthreads();
    fetch(base + kDsRows);
    for (int row = 0; row < n; ++row) {
      const float v_raw = v_lds[row][col_in];
      const float vv = CHANNEL ? v_raw : c_lds[row][1] * v_raw;
      const float g = CHANNEL ? 0.f : c_lds[row][0];
      float sum[2] = {0.f, 0.f};
#pragma unroll
      for (int i = 0; i < DS; ++i) {
        const int d = part * DS + i;
        S[i] = fmaf(k_lds[row][d], vv, (CHANNEL ? g_lds[CHANNEL ? row : 0][d] : g) * S[i]);
        sum[i % 2] = fmaf(S[i], q_lds[row][d], sum[i % 2]);
      }
      const float o = row_sum16(sum[0] + sum[1]);
      if (part == 0 && live)
        a.out[static_cast<int64_t>(row0 + base + row) * (a.H * Dv) + h * Dv + col] = CHANNEL ? o : fmaf(skip, v_raw, o);
    }
  }
#pragma unroll
  for (int i = 0; i < DS; ++i) {
    const int d = part * DS + i;
    if (live && d < D) s_ptr[static_cast<int64_t>(d) * Dv + col] = S[i];
  }
}

// A thread takes one channel and the up to 64 rows of a chunk.  R > 0: a middle of up to R, whose weights a thread keeps in
// registers; R == 0: any, in slices, with the rows' sums in registers.
constexpr int kGateSlice = 64;

// The logarithm of a decay.  In the running sums an absolute error of 1e-7 is what a float can hold anyway.
template <bool SUMS>
__device__ __forceinline__ float log_decay(float z, float inv_tau) {
  if (SUMS) return -(fmaxf(-z, 0.f) + __logf(1.0f + __expf(-fabsf(z)))) * inv_tau;
  return -softplus_f(-z) * inv_tau;
}

template <typename TW, int R, bool SUMS>
__global__ __launch_bounds__(kDsThreads) void decay_gates_kernel(const float* __restrict__ m, long long m_stride,
                                                                 const TW* __restrict__ w, const float* __restrict__ bias,
                                                                 float inv_tau, const int* __restrict__ seg_row0, int segments,
                                                                 float* __restrict__ out, int tokens, int rank, int channels) {
  constexpr int W = R > 0 ? R : kGateSlice;
  __shared__ __attribute__((aligned(16))) float ms[kChunkRows][W];
  ChunkAt at;
  if (SUMS) {
    at = find_chunk(seg_row0, segments, blockIdx.x);
  } else {
    at = ChunkAt{0, static_cast<int>(blockIdx.x) * kChunkRows, min(kChunkRows, tokens - static_cast<int>(blockIdx.x) * kChunkRows)};
  }
  if (at.rows <= 0) return;
  const int c = blockIdx.y * kDsThreads + threadIdx.x, cc = min(c, channels - 1);
  const float b = bias[cc];
  float sum = 0.f;
  auto finish = [&](int t, float z) {
    const float g = log_decay<SUMS>(z + b, inv_tau);
    sum += g;
    if (c < channels) out[static_cast<int64_t>(at.row0 + t) * channels + c] = SUMS ? sum : expf(g);
  };
  if constexpr (R > 0) {
    for (int i = threadIdx.x; i < at.rows * R; i += kDsThreads)
      ms[i / R][i % R] = i % R < rank ? m[(at.row0 + i / R) * m_stride + i % R] : 0.f;
    float wr[R];
#pragma unroll
    for (int r = 0; r < R; ++r) wr[r] = r < rank ? to_float(w[static_cast<int64_t>(cc) * rank + min(r, rank - 1)]) : 0.f;
    __syncthreads();
#pragma unroll 4
    for (int t = 0; t < at.rows; ++t) {
      float z = 0.f;
#pragma unroll
      for (int r = 0; r < R; ++r) z = fmaf(wr[r], ms[t][r], z);
      finish(t, z);
    }
  } else {
    float z[kChunkRows];
#pragma unroll
    for (int t = 0; t < kChunkRows; ++t) z[t] = 0.f;
    for (int r0 = 0; r0 < rank; r0 += kGateSlice) {
      const int n = min(kGateSlice, rank - r0);
      __syncthreads();                               // the slice before has been read
      for (int i = threadIdx.x; i < at.rows * n; i += kDsThreads) ms[i / n][i % n] = m[(at.row0 + i / n) * m_stride + r0 + i % n];
      __syncthreads();
      const TW* wr = w + static_cast<int64_t>(cc) * rank + r0;
      for (int r = 0; r < n; ++r) {
        const float wv = to_float(wr[r]);
#pragma unroll
        for (int t = 0; t < kChunkRows; ++t) z[t] = fmaf(wv, ms[t][r], z[t]);   // (rows past the chunk's: dropped below)
      }
    }
#pragma unroll
    for (int t = 0; t < kChunkRows; ++t)
      if (t < at.rows) finish(t, z[t]);
  }
}

// y [T, width] float32 times silu(z), each of `groups` equal runs of entries divided by its own root mean square, times a
// weight and a factor.  A workgroup a (row, group).
template <typename T>
__global__ __launch_bounds__(kDsThreads) void gated_norm_kernel(const float* __restrict__ y, const T* __restrict__ z,
                                                                long long z_stride, const float* __restrict__ w, float eps,
                                                                float factor, T* __restrict__ out, long long o_stride, int width,
                                                                int size) {
  extern __shared__ float xs[];
  __shared__ float red[kDsThreads / kWave];
  const int64_t t = blockIdx.x;
  const int first = blockIdx.y * size;
  float ss = 0.f;
  for (int i = threadIdx.x; i < size; i += kDsThreads) {
    const float x = y[t * width + first + i] * gate_act(to_float(z[t * z_stride + first + i]), kActSilu);
    xs[i] = x;
    ss = fmaf(x, x, ss);
  }
  const float inv = factor / sqrtf(block_sum<kDsThreads / kWave>(ss, red) / static_cast<float>(size) + eps);
  for (int i = threadIdx.x; i < size; i += kDsThreads)
    out[t * o_stride + first + i] = from_float<T>(xs[i] * inv * w[first + i]);
}

// A wave a (row, group), four entries a lane and access (sizes that are multiples of 4 up to 256 VPT, aligned rows).
template <typename T, int VPT>
__global__ __launch_bounds__(kDsThreads) void gated_norm_vec_kernel(const float* __restrict__ y, const T* __restrict__ z,
                                                                    long long z_stride, const float* __restrict__ w, float eps,
                                                                    float factor, T* __restrict__ out, long long o_stride,
                                                                    int width, int size, int64_t items) {
  const int64_t item = static_cast<int64_t>(blockIdx.x) * (kDsThreads / kWave) + threadIdx.x / kWave;
  if (item >= items) return;
  const int groups = width / size, lane = threadIdx.x % kWave;
  const int64_t t = item / groups;
  const int first = static_cast<int>(item % groups) * size;
  float4 x[VPT], g[VPT], wv[VPT];
#pragma unroll
  for (int j = 0; j < VPT; ++j) {
    const int i = first + min(4 * (lane + j * kWave), size - 4);
    x[j] = ld4<float>(y + t * width + i);
    g[j] = ld4<T>(z + t * z_stride + i);
    wv[j] = ld4<float>(w + i);
  }
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < VPT; ++j) {
    x[j] = float4{x[j].x * gate_act(g[j].x, kActSilu), x[j].y * gate_act(g[j].y, kActSilu), x[j].z * gate_act(g[j].z, kActSilu),
                  x[j].w * gate_act(g[j].w, kActSilu)};
    if (4 * (lane + j * kWave) < size) ss += (x[j].x * x[j].x + x[j].y * x[j].y) + (x[j].z * x[j].z + x[j].w * x[j].w);
  }
  const float inv = factor / sqrtf(wave_sum(ss) / static_cast<float>(size) + eps);
#pragma unroll
  for (int j = 0; j < VPT; ++j) {
    const int i = 4 * (lane + j * kWave);
    if (i < size)
      st4<T>(out + t * o_stride + first + i, float4{x[j].x * inv * wv[j].x, x[j].y * inv * wv[j].y, x[j].z * inv * wv[j].z,
                                                    x[j].w * inv * wv[j].w});
  }
}

}  // namespace arle

using namespace arle;

// q, k [T, G * D], v [T, H * Dv] of `dtype`, rows apart by their strides; out float32 [T, H * Dv].  channel: decay is
// [T, H * D] decays; else [T, H] raw step sizes with a_log, dt_bias, skip float32 [H].
extern "C" int arle_decay_scan(const void* q, long long q_stride, const void* k, long long k_stride, const void* v,
                               long long v_stride, int dtype, const float* decay, long long decay_stride, int channel,
                               const float* a_log, const float* dt_bias, const float* skip, float q_scale, float* s_state,
                               const int* seg_row0, const int* seg_slot, int segments, float* out, int H, int G, int D, int Dv,
                               void* stream) {
  if (segments == 0) return 0;
  if (H < 1 || H > 65535 || G < 1 || H % G || D < 1 || D > 256 || Dv < 1 || (!channel && (!a_log || !dt_bias || !skip)))
    return static_cast<int>(hipErrorInvalidValue);
  const ScanArgs a{q, q_stride, k, k_stride, v, v_stride, decay, decay_stride, a_log, dt_bias, skip, q_scale, s_state, seg_row0,
                   seg_slot, out, H, G, D, Dv};
  const dim3 grid(segments, H, (Dv + kDsCols - 1) / kDsCols);
  hipStream_t s = static_cast<hipStream_t>(stream);
#define ARLE_DS(T, DS)                                                                      \
  do {                                                                                      \
    if (channel) decay_scan_kernel<T, DS, true><<<grid, kDsThreads, 0, s>>>(a);             \
    else decay_scan_kernel<T, DS, false><<<grid, kDsThreads, 0, s>>>(a);                    \
  } while (0)
#define ARLE_DS_T(T) \
  if (D <= 32) ARLE_DS(T, 2); else if (D <= 64) ARLE_DS(T, 4); else if (D <= 128) ARLE_DS(T, 8); else ARLE_DS(T, 16)
  if (dtype == kF32) { ARLE_DS_T(float); } else { ARLE_DS_T(bf16); }
#undef ARLE_DS_T
#undef ARLE_DS
  return launch_status();
}

// m float32 [T, rank] (rows m_stride apart), w [channels, rank] of w_dtype, bias float32 [channels]; out float32
// [T, channels].  chunk_sums: the running sums of the decays' logarithms in every chunk of 64 rows of a segment (items: no
// fewer than there are chunks), else the decays.
extern "C" int arle_decay_gates(const float* m, long long m_stride, const void* w, int w_dtype, const float* bias, float inv_tau,
                                const int* seg_row0, int segments, int items, int chunk_sums, float* out, int tokens, int rank,
                                int channels, void* stream) {
  if (tokens == 0) return 0;
  const int blocks = chunk_sums ? items : (tokens + kChunkRows - 1) / kChunkRows;
  if (rank < 1 || channels < 1 || (channels + kDsThreads - 1) / kDsThreads > 65535 || blocks < 1)
    return static_cast<int>(hipErrorInvalidValue);
  const dim3 grid(blocks, (channels + kDsThreads - 1) / kDsThreads);
  hipStream_t s = static_cast<hipStream_t>(stream);
#define ARLE_DG(TW, R, SUMS)                                                                                               \
  decay_gates_kernel<TW, R, SUMS><<<grid, kDsThreads, 0, s>>>(m, m_stride, static_cast<const TW*>(w), bias, inv_tau, seg_row0, \
                                                              segments, out, tokens, rank, channels)
#define ARLE_DG_R(TW, SUMS)                    \
  do {                                         \
    if (rank <= 16) ARLE_DG(TW, 16, SUMS);     \
    else if (rank <= 64) ARLE_DG(TW, 64, SUMS);\
    else ARLE_DG(TW, 0, SUMS);                 \
  } while (0)
#define ARLE_DG_S(TW)                                            \
  do {                                                           \
    if (chunk_sums) ARLE_DG_R(TW, true); else ARLE_DG_R(TW, false); \
  } while (0)
  if (w_dtype == kF32) ARLE_DG_S(float); else ARLE_DG_S(bf16);
#undef ARLE_DG_S
#undef ARLE_DG_R
#undef ARLE_DG
  return launch_status();
}

// y float32 [T, width]; z, out [T, width] of `dtype` by their strides; w float32 [width]; groups divides width.
extern "C" int arle_gated_group_norm(const float* y, const void* z, long long z_stride, int dtype, const float* w, float eps,
                                     float factor, void* out, long long o_stride, int tokens, int width, int groups,
                                     void* stream) {
  if (tokens == 0) return 0;
  if (width < 1 || groups < 1 || width % groups || groups > 65535 || width / groups > 16384)
    return static_cast<int>(hipErrorInvalidValue);
  const int size = width / groups;
  const dim3 grid(tokens, groups);
  const auto al = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  if (size % 4 == 0 && size <= 2048 && width % 4 == 0 && z_stride % 4 == 0 && o_stride % 4 == 0 && al(y) && al(w) &&
      reinterpret_cast<uintptr_t>(z) % (dtype == kF32 ? 16 : 8) == 0 && reinterpret_cast<uintptr_t>(out) % (dtype == kF32 ? 16 : 8) == 0) {
    const int64_t items = static_cast<int64_t>(tokens) * groups;
    const unsigned blocks = static_cast<unsigned>((items + kDsThreads / kWave - 1) / (kDsThreads / kWave));
    hipStream_t s = static_cast<hipStream_t>(stream);
#define ARLE_GNV(T, VPT)                                                                                                   \
  gated_norm_vec_kernel<T, VPT><<<blocks, kDsThreads, 0, s>>>(y, static_cast<const T*>(z), z_stride, w, eps, factor,       \
                                                              static_cast<T*>(out), o_stride, width, size, items)
#define ARLE_GNV_T(T)                        \
  do {                                       \
    if (size <= 256) ARLE_GNV(T, 1);         \
    else if (size <= 512) ARLE_GNV(T, 2);    \
    else if (size <= 1024) ARLE_GNV(T, 4);   \
    else ARLE_GNV(T, 8);                     \
  } while (0)
    if (dtype == kF32) ARLE_GNV_T(float); else ARLE_GNV_T(bf16);
#undef ARLE_GNV_T
#undef ARLE_GNV
    return launch_status();
  }
  const size_t lds = static_cast<size_t>(size) * sizeof(float);     // at most 64 KB
  static bool raised = false;
  if (!raised && lds > 48 * 1024) {
    const void* kernels[] = {reinterpret_cast<const void*>(&gated_norm_kernel<float>),
                             reinterpret_cast<const void*>(&gated_norm_kernel<bf16>)};
    for (const void* f : kernels) {
      const hipError_t e = hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, 64 * 1024);
      if (e != hipSuccess) return static_cast<int>(e);
    }
    raised = true;
  }
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (dtype == kF32)
    gated_norm_kernel<float><<<grid, kDsThreads, lds, s>>>(y, static_cast<const float*>(z), z_stride, w, eps, factor,
                                                                 static_cast<float*>(out), o_stride, width, size);
  else
    gated_norm_kernel<bf16><<<grid, kDsThreads, lds, s>>>(y, static_cast<const bf16*>(z), z_stride, w, eps, factor,
                                                                static_cast<bf16*>(out), o_stride, width, size);
  return launch_status();
}
