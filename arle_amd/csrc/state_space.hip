// A state-space layer with one decay a head and token, for the rows of a packed step, continued across steps through a
// per-request state S [heads, N, P] in 32-bit floats and the last taps - 1 inputs of its short convolution.
//
//   dt = softplus(raw + dt_bias_h),  S_t = exp(-exp(A_log_h) dt_t) S_(t-1) + dt_t B_t x_t^T,  y_t = S_t^T C_t + D_h x_t
//   (x [H, P]; B, C [G, N], head h reads group h / (H / G); all three behind the convolution and its silu, in bfloat16)
//
// Two forms beside the one row by row in decay_scan.hip, both for bfloat16 engines:
//   * a decoded row: `state_space_decode` goes from the partial sums of the input projection (columns z | x | B | C | dt) to
//     y silu(z), with the convolution on the way; `state_space_finish` norms that in groups and moves the convolution's
//     inputs on (in a kernel of its own, because every head of a group reads the old ones).
//   * chunks of 64 rows on the matrix cores.  With L_i the sum of the decays' logarithms over the chunk's rows up to i, and S_0
//     the state in front of a chunk of n rows:
//       y_i = exp(L_i) S_0^T C_i + sum_(j<=i) M_ij x_j + D x_i,    M_ij = (C_i . B_j) exp(L_i - L_j) dt_j
//       S_n = exp(L_(n-1)) S_0 + sum_j exp(L_(n-1) - L_j) dt_j B_j x_j^T
//     One kernel makes every chunk's own sum, one carries the state over the chunks, one makes the outputs.  x, B and C are
//     bfloat16 numbers, so every product has an operand that is one exactly; the other, 32-bit, operand (M, the state, the
//     counted x) goes in as three bfloat16 numbers that add up to it (24 bits), and the sums are 32-bit.
#include "chunks.h"
#include "lane_sums.h"

namespace arle {

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef float f32x4_t __attribute__((ext_vector_type(4)));
typedef uint32_t u32x4_t __attribute__((ext_vector_type(4)));

constexpr int kSsThreads = 256;
constexpr int kSsWaves = kSsThreads / kWave;

__device__ __forceinline__ float as_bf16(float v) { return to_float(from_float<bf16>(v)); }
__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }

// ---- a decoded row ---------------------------------------------------------------------------------
constexpr int kSsMaxN = 256, kSsMaxP = 256, kSsMaxTaps = 16;
constexpr int kSsFlight = 8;   // rows of S a thread has in flight

struct SsDecodeArgs {
  const float* y; int parts; long long part_stride, row_stride;   // columns z | x | B | C | dt of the projection's sums
  const void* conv; int conv_dtype; const void* conv_bias; int cb_dtype; const bf16* conv_state; int taps;
  const float* a_log; const float* dt_bias; const float* skip;
  const int* seg_row0; const int* seg_slot;
  float* s_state;
  float* out;                                                     // [T, H * P]: y silu(z)
  int H, G, N, P;
};

// One workgroup a (request, head).  A thread holds four columns of S and walks rows of it, RP rows a pass.
__global__ __launch_bounds__(kSsThreads) void state_space_decode_kernel(const SsDecodeArgs a) {
  __shared__ __attribute__((aligned(16))) float u[kSsMaxP + 2 * kSsMaxN];    // x, B, C behind the convolution
  __shared__ __attribute__((aligned(16))) float os[4 * kSsThreads];          // partial read-outs, [pass row][P]
  __shared__ float zs[kSsMaxP];
  __shared__ float dt_s;
  const int h = blockIdx.y, tid = threadIdx.x, P = a.P, N = a.N;
  const int64_t t = a.seg_row0[blockIdx.x], slot = a.seg_slot[blockIdx.x];
  const int grp = h / (a.H / a.G), inner = a.H * P, channels = inner + 2 * a.G * N;
  const int per_row = P / 4, RP = kSsThreads / per_row;
  const int rp = tid / per_row, c = 4 * (tid % per_row);
  const bool mine = rp < RP;
  float* s_ptr = a.s_state + (slot * a.H + h) * N * P;
  float4 next[kSsFlight];
  auto fetch = [&](int d0) {   // rows past N fetch the last row again and are dropped
#pragma unroll
    for (int i = 0; i < kSsFlight; ++i) next[i] = ld4<float>(s_ptr + static_cast<int64_t>(min(d0 + i * RP, N - 1)) * P + c);
  };
  fetch(min(rp, RP - 1));
  const float* yr = a.y + t * a.row_stride;
  for (int i = tid; i < P + 2 * N; i += kSsThreads) {
    const int ch = i < P ? h * P + i : (i < P + N ? inner + grp * N + i - P : inner + (a.G + grp) * N + i - P - N);
    const float now = as_bf16(sum_parts(yr + inner + ch, a.parts, a.part_stride));
    float acc = fmaf(load_as_float(a.conv, a.conv_dtype, static_cast<int64_t>(ch) * a.taps + a.taps - 1), now,
                     load_as_float(a.conv_bias, a.cb_dtype, ch));
    for (int back = 1; back < a.taps; ++back)
      acc = fmaf(load_as_float(a.conv, a.conv_dtype, static_cast<int64_t>(ch) * a.taps + a.taps - 1 - back),
                 to_float(a.conv_state[(slot * (a.taps - 1) + a.taps - 1 - back) * channels + ch]), acc);
    u[i] = as_bf16(silu_f(acc));
  }
  for (int i = tid; i < P; i += kSsThreads) zs[i] = as_bf16(sum_parts(yr + h * P + i, a.parts, a.part_stride));
  if (tid == 0) dt_s = softplus_f(sum_parts(yr + inner + channels + h, a.parts, a.part_stride) + a.dt_bias[h]);
  __syncthreads();
  const float dt = dt_s, keep = expf(-expf(a.a_log[h]) * dt);
  const float4 x4 = *reinterpret_cast<const float4*>(&u[c]);
  const float4 v4 = {dt * x4.x, dt * x4.y, dt * x4.z, dt * x4.w};
  float4 o = {0.f, 0.f, 0.f, 0.f};
  if (mine) {
    for (int d0 = rp; d0 < N; d0 += kSsFlight * RP) {
      float4 now[kSsFlight];
#pragma unroll
      for (int i = 0; i < kSsFlight; ++i) now[i] = next[i];
      if (d0 + kSsFlight * RP < N) fetch(d0 + kSsFlight * RP);
#pragma unroll
      for (int i = 0; i < kSsFlight; ++i) {
        const int d = d0 + i * RP;
        if (d < N) {
          const float bd = u[P + d], cd = u[P + N + d];
          float4 s = now[i];
          s.x = fmaf(bd, v4.x, keep * s.x); s.y = fmaf(bd, v4.y, keep * s.y);
          s.z = fmaf(bd, v4.z, keep * s.z); s.w = fmaf(bd, v4.w, keep * s.w);
          o.x = fmaf(cd, s.x, o.x); o.y = fmaf(cd, s.y, o.y); o.z = fmaf(cd, s.z, o.z); o.w = fmaf(cd, s.w, o.w);
          st4<float>(s_ptr + static_cast<int64_t>(d) * P + c, s);
        }
      }
    }
    *reinterpret_cast<float4*>(&os[rp * P + c]) = o;
  }
  __syncthreads();
  for (int e = tid; e < P; e += kSsThreads) {
    float sum = 0.f;
    for (int p = 0; p < RP; ++p) sum += os[p * P + e];
    a.out[t * inner + h * P + e] = fmaf(a.skip[h], u[e], sum) * silu_f(zs[e]);
  }
}

// Decoded rows: workgroups y < norm_groups norm a group of `yv` (which holds y silu(z)) into out; the others move the
// convolution's inputs on, 256 channels each.
__global__ __launch_bounds__(kSsThreads) void state_space_finish_kernel(
    const float* __restrict__ yv, const float* __restrict__ w, float eps, float factor, bf16* __restrict__ out, long long o_stride,
    int width, int norm_groups, const float* __restrict__ y, int parts, long long part_stride, long long row_stride,
    bf16* __restrict__ conv_state, int taps, int channels, const int* __restrict__ seg_row0, const int* __restrict__ seg_slot) {
  __shared__ float red[kSsWaves];
  const int64_t t = seg_row0[blockIdx.x];
  if (static_cast<int>(blockIdx.y) < norm_groups) {
    const int size = width / norm_groups, first = blockIdx.y * size;
    const float* row = yv + t * width + first;
    float ss = 0.f;
    for (int i = threadIdx.x; i < size; i += kSsThreads) ss = fmaf(row[i], row[i], ss);
    const float inv = factor / sqrtf(block_sum<kSsWaves>(ss, red) / static_cast<float>(size) + eps);
    for (int i = threadIdx.x; i < size; i += kSsThreads) out[t * o_stride + first + i] = from_float<bf16>(row[i] * inv * w[first + i]);
    return;
  }
  const int c = (blockIdx.y - norm_groups) * kSsThreads + threadIdx.x;
  if (c >= channels) return;
  const float now = sum_parts(y + t * row_stride + width + c, parts, part_stride);
  bf16* st = conv_state + static_cast<int64_t>(seg_slot[blockIdx.x]) * (taps - 1) * channels + c;
  for (int j = 0; j + 1 < taps - 1; ++j) st[static_cast<int64_t>(j) * channels] = st[static_cast<int64_t>(j + 1) * channels];
  st[static_cast<int64_t>(taps - 2) * channels] = from_float<bf16>(now);
}

// ---- chunks of rows on the matrix cores ------------------------------------------------------------
// `v_mfma_f32_16x16x32_bf16`: both operands are eight consecutive k a lane (row or column lane % 16, k from 8 (lane / 16)
// on), the result's lane holds rows 4 (lane / 16) .. + 3 of column lane % 16.
// Tiles in LDS are rows of pieces of eight bfloat16; a row's pieces are permuted within every eight of them by the row's
// number, so that neither the sixteen rows of an operand nor the columns that a transposing write goes through share banks.
struct SsChunkArgs {
  const bf16* u; long long u_stride;                     // x | B | C behind the convolution
  const float* dt; long long dt_stride;                  // [T, H] raw step sizes
  const float* a_log; const float* dt_bias; const float* skip;
  const int* seg_row0; const int* seg_slot; int segments;
  float* s_state;
  float* work;                                           // [items, H, P, N]: a chunk's own sum, then the state in front of it
  float* ends;                                           // [items, H]: L behind the chunk's last row
  float* out;                                            // [T, H * P]
  int H, G, N, P;
};

__device__ __forceinline__ int piece_at(int row, int piece) { return (piece & ~7) | ((piece ^ (row + (row >> 3))) & 7); }

struct RowDecay {
  float dt, hi, lo;      // of the lane's row: the step size, and L as two numbers (differences of large L count)
};
// Lane j looks after row j of the chunk (rows past its end: a step of size zero).
__device__ __forceinline__ RowDecay row_decay(const SsChunkArgs& a, const ChunkAt& at, int h, int lane) {
  const float raw = a.dt[static_cast<int64_t>(at.row0 + min(lane, at.rows - 1)) * a.dt_stride + h];
  const float dt = lane < at.rows ? softplus_f(raw + a.dt_bias[h]) : 0.f;
  double sum = -static_cast<double>(expf(a.a_log[h])) * dt;
#pragma unroll
  for (int off = 1; off < kWave; off <<= 1) {
    const double before = __shfl_up(sum, off, kWave);
    if (lane >= off) sum += before;
  }
  const float hi = static_cast<float>(sum);
  return RowDecay{dt, hi, static_cast<float>(sum - hi)};
}

// v = hi + mid + lo, bits of bfloat16 each.
__device__ __forceinline__ void split3(float v, uint16_t& hi, uint16_t& mid, uint16_t& lo) {
  hi = f32_to_bf16_bits(v);
  const float r1 = v - __uint_as_float(static_cast<uint32_t>(hi) << 16);
  mid = f32_to_bf16_bits(r1);
  lo = f32_to_bf16_bits(r1 - __uint_as_float(static_cast<uint32_t>(mid) << 16));
}
__device__ __forceinline__ uint32_t pair(uint16_t a, uint16_t b) { return a | (static_cast<uint32_t>(b) << 16); }

// Eight 32-bit numbers as three operands.
__device__ __forceinline__ void split8(const float4& lo4, const float4& hi4, bf16x8_t (&op)[3]) {
  const float v[8] = {lo4.x, lo4.y, lo4.z, lo4.w, hi4.x, hi4.y, hi4.z, hi4.w};
  u32x4_t w[3];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    uint16_t a[3], b[3];
    split3(v[2 * i], a[0], a[1], a[2]);
    split3(v[2 * i + 1], b[0], b[1], b[2]);
#pragma unroll
    for (int s = 0; s < 3; ++s) w[s][i] = pair(a[s], b[s]);
  }
#pragma unroll
  for (int s = 0; s < 3; ++s) op[s] = __builtin_bit_cast(bf16x8_t, w[s]);
}

__device__ __forceinline__ bf16x8_t operand(const bf16* tile, int row, int row_pieces, int piece) {
  return __builtin_bit_cast(bf16x8_t, *reinterpret_cast<const u32x4_t*>(tile + (row * row_pieces + piece_at(row, piece)) * 8));
}

// Columns first .. first + 8 count - 1 of the chunk's rows turned: tile[column][64 rows].  Eight rows of eight columns a
// thread and time; rows past the chunk's end and columns from `width` on are zero.
__device__ __forceinline__ void stage_turned(const bf16* src, long long stride, int rows, int width, int count, bf16* tile, int tid) {
  for (int i = tid; i < 8 * count; i += kSsThreads) {
    const int nb = i % count, jb = i / count, col = min(8 * nb, width - 8);
    u32x4_t in[8];
#pragma unroll
    for (int r = 0; r < 8; ++r) in[r] = *reinterpret_cast<const u32x4_t*>(src + static_cast<int64_t>(min(8 * jb + r, rows - 1)) * stride + col);
    const bool live = 8 * nb < width;
#pragma unroll
    for (int c = 0; c < 8; ++c) {
      u32x4_t o;
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        const uint32_t lo = in[2 * k][c / 2] >> (16 * (c % 2)) & 0xffffu, hi = in[2 * k + 1][c / 2] >> (16 * (c % 2)) & 0xffffu;
        o[k] = (live && 8 * jb + 2 * k < rows ? lo : 0u) | (live && 8 * jb + 2 * k + 1 < rows ? hi << 16 : 0u);
      }
      const int row = 8 * nb + c;
      *reinterpret_cast<u32x4_t*>(tile + (row * 8 + piece_at(row, jb)) * 8) = o;
    }
  }
}

constexpr int kSsTurned = 64;      // columns of x turned at a time by the first kernel

// U^T of a chunk: work[item, h, p, n] = sum_j exp(L_(n-1) - L_j) dt_j x_j[p] B_j[n].
__global__ __launch_bounds__(kSsThreads) void state_space_chunk_sum_kernel(const SsChunkArgs a) {
  extern __shared__ __attribute__((aligned(16))) bf16 tiles[];
  __shared__ float count[kChunkRows];
  const ChunkAt at = find_chunk(a.seg_row0, a.segments, blockIdx.x);
  if (at.rows == 0) return;
  const int h = blockIdx.y, tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, n = lane % 16, g = lane / 16;
  const int N = a.N, P = a.P, NB = (N + 15) / 16 * 2, inner = a.H * P, grp = h / (a.H / a.G);
  bf16* bt = tiles;                                  // [16 * ceil(N / 16)][64 rows]
  bf16* xt = tiles + 8 * NB * kChunkRows;            // three of [64 columns][64 rows]
  const bf16* u0 = a.u + static_cast<int64_t>(at.row0) * a.u_stride;
  stage_turned(u0 + inner + grp * N, a.u_stride, at.rows, N, NB, bt, tid);
  {
    const RowDecay r = row_decay(a, at, h, lane);
    const float end = __shfl(r.hi, kWave - 1, kWave), end_lo = __shfl(r.lo, kWave - 1, kWave);
    if (wave == 0) {
      count[lane] = expf((end - r.hi) + (end_lo - r.lo)) * r.dt;
      if (lane == 0) a.ends[static_cast<int64_t>(blockIdx.x) * a.H + h] = end;
    }
  }
  float* dst = a.work + (static_cast<int64_t>(blockIdx.x) * a.H + h) * N * P;
  for (int p0 = 0; p0 < P; p0 += kSsTurned) {
    const int pairs = min(kSsTurned, P - p0) / 2;
    __syncthreads();                                 // the numbers are there; the columns before have been read
    for (int i = tid; i < 8 * kSsTurned / 2; i += kSsThreads) {      // eight rows of two columns a thread
      const int pp = i % (kSsTurned / 2), jb = i / (kSsTurned / 2), col = h * P + p0 + 2 * min(pp, pairs - 1);
      uint32_t in[8];
#pragma unroll
      for (int r = 0; r < 8; ++r) in[r] = *reinterpret_cast<const uint32_t*>(u0 + static_cast<int64_t>(min(8 * jb + r, at.rows - 1)) * a.u_stride + col);
      u32x4_t o[2][3];
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        const float f0 = pp < pairs ? count[8 * jb + 2 * k] : 0.f, f1 = pp < pairs ? count[8 * jb + 2 * k + 1] : 0.f;
#pragma unroll
        for (int c = 0; c < 2; ++c) {
          const float v0 = c ? __uint_as_float(in[2 * k] & 0xffff0000u) : __uint_as_float(in[2 * k] << 16);
          const float v1 = c ? __uint_as_float(in[2 * k + 1] & 0xffff0000u) : __uint_as_float(in[2 * k + 1] << 16);
          uint16_t s0[3], s1[3];
          split3(f0 * v0, s0[0], s0[1], s0[2]);
          split3(f1 * v1, s1[0], s1[1], s1[2]);
#pragma unroll
          for (int s = 0; s < 3; ++s) o[c][s][k] = pair(s0[s], s1[s]);
        }
      }
#pragma unroll
      for (int c = 0; c < 2; ++c) {
        const int row = 2 * pp + c;
#pragma unroll
        for (int s = 0; s < 3; ++s) *reinterpret_cast<u32x4_t*>(xt + ((s * kSsTurned + row) * 8 + piece_at(row, jb)) * 8) = o[c][s];
      }
    }
    __syncthreads();
    for (int n0 = 16 * wave; n0 < N; n0 += 16 * kSsWaves) {
      f32x4_t acc[kSsTurned / 16];
#pragma unroll
      for (int j = 0; j < kSsTurned / 16; ++j) acc[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const bf16x8_t b = operand(bt, n0 + n, 8, 4 * k + g);
#pragma unroll
        for (int j = 0; j < kSsTurned / 16; ++j)
#pragma unroll
          for (int s = 2; s >= 0; --s)
            acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(b, operand(xt + s * kSsTurned * kChunkRows, 16 * j + n, 8, 4 * k + g), acc[j], 0, 0, 0);
      }
      // acc[j]: state rows n0 + 4 g .. + 3 of column p0 + 16 j + n
#pragma unroll
      for (int j = 0; j < kSsTurned / 16; ++j) {
        const int p = p0 + 16 * j + n, d = n0 + 4 * g;
        if (p < P && d < N) st4<float>(dst + static_cast<int64_t>(p) * N + d, float4{acc[j][0], acc[j][1], acc[j][2], acc[j][3]});
      }
    }
  }
}

// The state carried over a request's chunks: work becomes the state in front of each chunk, s_state the one behind the
// last.  A thread takes four entries of one column p.
constexpr int kSsCarryFlight = 8;

__global__ __launch_bounds__(kSsThreads) void state_space_chunk_carry_kernel(const SsChunkArgs a) {
  const int seg = blockIdx.x, h = blockIdx.y, N = a.N, P = a.P;
  const int i = blockIdx.z * kSsThreads + threadIdx.x;
  if (i >= N / 4 * P) return;
  const int p = i / (N / 4), d = 4 * (i % (N / 4));
  int first = 0;
  for (int s = 0; s < seg; ++s) first += (a.seg_row0[s + 1] - a.seg_row0[s] + kChunkRows - 1) / kChunkRows;
  const int chunks = (a.seg_row0[seg + 1] - a.seg_row0[seg] + kChunkRows - 1) / kChunkRows;
  if (chunks == 0) return;
  float* st = a.s_state + (static_cast<int64_t>(a.seg_slot[seg]) * a.H + h) * N * P + static_cast<int64_t>(d) * P + p;
  float4 S = {st[0], st[P], st[2 * P], st[3 * P]};
  const int64_t step = static_cast<int64_t>(a.H) * N * P;
  float* w = a.work + (static_cast<int64_t>(first) * a.H + h) * N * P + static_cast<int64_t>(p) * N + d;
  const float* ends = a.ends + static_cast<int64_t>(first) * a.H + h;
  for (int c0 = 0; c0 < chunks; c0 += kSsCarryFlight) {
    float4 u[kSsCarryFlight];
    float f[kSsCarryFlight];
#pragma unroll
    for (int j = 0; j < kSsCarryFlight; ++j) {
      const int c = min(c0 + j, chunks - 1);
      u[j] = ld4<float>(w + c * step);
      f[j] = ends[static_cast<int64_t>(c) * a.H];
    }
#pragma unroll
    for (int j = 0; j < kSsCarryFlight; ++j) {
      if (c0 + j < chunks) {
        st4<float>(w + (c0 + j) * step, S);
        const float e = expf(f[j]);
        S = float4{fmaf(e, S.x, u[j].x), fmaf(e, S.y, u[j].y), fmaf(e, S.z, u[j].z), fmaf(e, S.w, u[j].w)};
      }
    }
  }
  st[0] = S.x; st[P] = S.y; st[2 * P] = S.z; st[3 * P] = S.w;
}

// The outputs of a chunk.  Wave w makes the rows 16 w .. + 15 of M, then all rows of the columns 16 (w + 4 j) .. + 15, j < NT.
template <int NT>
__global__ __launch_bounds__(kSsThreads) void state_space_chunk_out_kernel(const SsChunkArgs a) {
  extern __shared__ __attribute__((aligned(16))) bf16 tiles[];
  __shared__ float Ls[kChunkRows], Ls_lo[kChunkRows], dts[kChunkRows];
  const ChunkAt at = find_chunk(a.seg_row0, a.segments, blockIdx.x);
  if (at.rows == 0) return;
  const int h = blockIdx.y, tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, n = lane % 16, g = lane / 16;
  const int N = a.N, P = a.P, NP = (N + 63) / 64 * 8, inner = a.H * P, grp = h / (a.H / a.G);     // NP: pieces of a row of C
  bf16* ct = tiles;                                  // C, [64][8 NP]
  bf16* xt = ct + kChunkRows * 8 * NP;               // x turned, [64 NT columns][64 rows]
  bf16* bt = xt + 64 * NT * kChunkRows;              // B, [64][8 NP]; then M as three of [64][64]
  const bf16* u0 = a.u + static_cast<int64_t>(at.row0) * a.u_stride;
  const float* S0 = a.work + (static_cast<int64_t>(blockIdx.x) * a.H + h) * N * P;               // [p][n]
  const u32x4_t zero = {0, 0, 0, 0};
  for (int i = tid; i < kChunkRows * NP; i += kSsThreads) {
    const int r = i / NP, c = i % NP;
    const bf16* row = u0 + static_cast<int64_t>(min(r, at.rows - 1)) * a.u_stride + inner + grp * N + min(8 * c, N - 8);
    const u32x4_t b = *reinterpret_cast<const u32x4_t*>(row), cc = *reinterpret_cast<const u32x4_t*>(row + a.G * N);
    const bool in = r < at.rows && 8 * c < N;
    const int at8 = (r * NP + piece_at(r, c)) * 8;
    *reinterpret_cast<u32x4_t*>(bt + at8) = in ? b : zero;
    *reinterpret_cast<u32x4_t*>(ct + at8) = in ? cc : zero;
  }
  stage_turned(u0 + h * P, a.u_stride, at.rows, P, 8 * NT, xt, tid);
  if (wave == 0) {
    const RowDecay r = row_decay(a, at, h, lane);
    Ls[lane] = r.hi;
    Ls_lo[lane] = r.lo;
    dts[lane] = r.dt;
  }
  __syncthreads();
  f32x4_t m[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) m[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int k = 0; k < NP / 4; ++k) {
    const bf16x8_t c = operand(ct, 16 * wave + n, NP, 4 * k + g);
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j <= wave) m[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(c, operand(bt, 16 * j + n, NP, 4 * k + g), m[j], 0, 0, 0);
  }
  // exp(L_i) S_0^T C_i: each wave reads its own columns of the state
  f32x4_t o[4][NT];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < NT; ++j) o[i][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
  for (int k = 0; k < NP / 4; ++k) {                 // (past N the rows of C are zero)
    bf16x8_t c[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) c[i] = operand(ct, 16 * i + n, NP, 4 * k + g);
#pragma unroll
    for (int j = 0; j < NT; ++j) {
      const float* s = S0 + static_cast<int64_t>(min(16 * (wave + 4 * j) + n, P - 1)) * N + min(32 * k + 8 * g, N - 8);
      bf16x8_t op[3];
      split8(ld4<float>(s), ld4<float>(s + 4), op);
#pragma unroll
      for (int s3 = 2; s3 >= 0; --s3)
#pragma unroll
        for (int i = 0; i < 4; ++i) o[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(c[i], op[s3], o[i][j], 0, 0, 0);
    }
  }
  __syncthreads();                                   // B has been read by every wave
  bf16* mt = bt;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    if (j > (wave | 1)) continue;                    // what no product reads
    const int col = 16 * j + n;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int row = 16 * wave + 4 * g + i;
      const float v = col <= row ? m[j][i] * expf((Ls[row] - Ls[col]) + (Ls_lo[row] - Ls_lo[col])) * dts[col] : 0.f;
      uint16_t s3[3];
      split3(v, s3[0], s3[1], s3[2]);
#pragma unroll
      for (int s = 0; s < 3; ++s) mt[((s * kChunkRows + row) * 8 + piece_at(row, col / 8)) * 8 + col % 8].bits = s3[s];
    }
  }
  const float skip = a.skip[h];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float f = expf(Ls[16 * i + 4 * g + e]);
#pragma unroll
      for (int j = 0; j < NT; ++j) o[i][j][e] *= f;
    }
  __syncthreads();
#pragma unroll
  for (int k = 0; k < 2; ++k) {
    bf16x8_t x[NT];
#pragma unroll
    for (int j = 0; j < NT; ++j) x[j] = operand(xt, 16 * (wave + 4 * j) + n, 8, 4 * k + g);
#pragma unroll
    for (int s = 2; s >= 0; --s)
#pragma unroll
      for (int i = 2 * k; i < 4; ++i) {
        const bf16x8_t mo = operand(mt + s * kChunkRows * kChunkRows, 16 * i + n, 8, 4 * k + g);
#pragma unroll
        for (int j = 0; j < NT; ++j) o[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(mo, x[j], o[i][j], 0, 0, 0);
      }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < NT; ++j) {
      const int p = 16 * (wave + 4 * j) + n, r0 = 16 * i + 4 * g;
      if (p >= P) continue;
      const uint2 xr = *reinterpret_cast<const uint2*>(xt + (p * 8 + piece_at(p, r0 / 8)) * 8 + r0 % 8);
      const float x[4] = {__uint_as_float(xr.x << 16), __uint_as_float(xr.x & 0xffff0000u), __uint_as_float(xr.y << 16),
                          __uint_as_float(xr.y & 0xffff0000u)};
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (r0 + e < at.rows) a.out[static_cast<int64_t>(at.row0 + r0 + e) * inner + h * P + p] = fmaf(skip, x[e], o[i][j][e]);
    }
}

}  // namespace arle

using namespace arle;

// y float32: `parts` partial products part_stride apart of rows row_stride apart, columns z | x | B | C | dt; one row a
// segment.  conv [channels, taps] and conv_bias [channels] of their types; conv_state bfloat16 [slots, taps - 1, channels] (null
// with one tap).  yv: float32 [T, H * P] scratch; norm float32 [H * P]; out bfloat16 [T, H * P], rows o_stride apart.
extern "C" int arle_state_space_decode(const float* y, int parts, long long part_stride, long long row_stride, const void* conv,
                                       int conv_dtype, const void* conv_bias, int cb_dtype, void* conv_state, int taps,
                                       const float* a_log, const float* dt_bias, const float* skip, const int* seg_row0,
                                       const int* seg_slot, float* s_state, float* yv, const float* norm, float eps, float factor,
                                       int norm_groups, void* out, long long o_stride, int segments, int H, int G, int N, int P,
                                       void* stream) {
  if (segments == 0) return 0;
  if (parts < 1 || H < 1 || H > 65535 || G < 1 || H % G || N < 1 || N > kSsMaxN || P < 4 || P > kSsMaxP || P % 4 || taps < 1 ||
      taps > kSsMaxTaps || (taps > 1 && !conv_state) || norm_groups < 1 || (H * P) % norm_groups ||
      reinterpret_cast<uintptr_t>(s_state) % 16)
    return static_cast<int>(hipErrorInvalidValue);
  hipStream_t s = static_cast<hipStream_t>(stream);
  const SsDecodeArgs a{y, parts, part_stride, row_stride, conv, conv_dtype, conv_bias, cb_dtype, static_cast<const bf16*>(conv_state),
                       taps, a_log, dt_bias, skip, seg_row0, seg_slot, s_state, yv, H, G, N, P};
  state_space_decode_kernel<<<dim3(segments, H), kSsThreads, 0, s>>>(a);
  const int channels = H * P + 2 * G * N, moves = taps > 1 ? (channels + kSsThreads - 1) / kSsThreads : 0;
  if (norm_groups + moves > 65535) return static_cast<int>(hipErrorInvalidValue);
  state_space_finish_kernel<<<dim3(segments, norm_groups + moves), kSsThreads, 0, s>>>(
      yv, norm, eps, factor, static_cast<bf16*>(out), o_stride, H * P, norm_groups, y, parts, part_stride, row_stride,
      static_cast<bf16*>(conv_state), taps, channels, seg_row0, seg_slot);
  return launch_status();
}

// u bfloat16 [T, x | B | C], rows u_stride apart; dt float32 [T, >= H].  work float32 [items, H, P, N] and ends float32
// [items, H] with items at least the number of chunks of 64 rows of all segments.  out float32 [T, H * P].
extern "C" int arle_state_space_chunks(const void* u, long long u_stride, const float* dt, long long dt_stride, const float* a_log,
                                       const float* dt_bias, const float* skip, const int* seg_row0, const int* seg_slot,
                                       int segments, int items, float* s_state, float* work, float* ends, float* out, int H, int G,
                                       int N, int P, void* stream) {
  if (segments == 0 || items == 0) return 0;
  auto al = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  if (H < 1 || H > 65535 || G < 1 || H % G || N < 8 || N > 256 || N % 8 || P < 8 || P > 256 || P % 8 || u_stride % 8 || !al(u) ||
      !al(work))
    return static_cast<int>(hipErrorInvalidValue);
  const SsChunkArgs a{static_cast<const bf16*>(u), u_stride, dt, dt_stride, a_log, dt_bias, skip, seg_row0, seg_slot, segments,
                      s_state, work, ends, out, H, G, N, P};
  hipStream_t s = static_cast<hipStream_t>(stream);
  const int nt = P <= 64 ? 1 : (P <= 128 ? 2 : 4), np = (N + 63) / 64 * 64;
  const size_t sum_lds = static_cast<size_t>(kChunkRows) * ((N + 15) / 16 * 16 + 3 * kSsTurned) * sizeof(bf16);
  const size_t out_lds = static_cast<size_t>(kChunkRows) * (np + 64 * nt + max(np, 3 * kChunkRows)) * sizeof(bf16);
  static bool raised = false;
  if (!raised) {
    const void* kernels[] = {reinterpret_cast<const void*>(&state_space_chunk_sum_kernel),
                             reinterpret_cast<const void*>(&state_space_chunk_out_kernel<1>),
                             reinterpret_cast<const void*>(&state_space_chunk_out_kernel<2>),
                             reinterpret_cast<const void*>(&state_space_chunk_out_kernel<4>)};
    for (const void* f : kernels) {
      const hipError_t e = hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024);
      if (e != hipSuccess) return static_cast<int>(e);
    }
    raised = true;
  }
  const dim3 grid(items, H);
  state_space_chunk_sum_kernel<<<grid, kSsThreads, sum_lds, s>>>(a);
  state_space_chunk_carry_kernel<<<dim3(segments, H, (N / 4 * P + kSsThreads - 1) / kSsThreads), kSsThreads, 0, s>>>(a);
  if (nt == 1)
    state_space_chunk_out_kernel<1><<<grid, kSsThreads, out_lds, s>>>(a);
  else if (nt == 2)
    state_space_chunk_out_kernel<2><<<grid, kSsThreads, out_lds, s>>>(a);
  else
    state_space_chunk_out_kernel<4><<<grid, kSsThreads, out_lds, s>>>(a);
  return launch_status();
}
