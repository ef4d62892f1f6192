// Retention: linear attention with one fixed decay a head and no softmax, for the rows of a packed step, continued
// across steps through a per-request state S [heads, D, Dv] in 32-bit floats.
//
//   q, k turn by their position's angles (the first `rot` entries, entry i with i + rot / 2);  k <- k * D^(-1/2)
//   S_t = g_h S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t,   y_t = o_t / sqrt(mean(o_t^2) + eps) * silu(gate_t)   (per head)
//
// Three ways to the same numbers, all in 32-bit arithmetic from the projections' 32-bit sums on:
//   * row by row (`retention_prep`, `retention_scan`, `retention_output`): every sum in one order whatever a step holds;
//   * a decoded row (`retention_decode`): one kernel from the product's partial sums to y, the state read and written
//     once in whole lines;
//   * chunks of 64 rows on the matrix cores' float32 products (`retention_chunks`).  With i, j rows of a chunk of n rows
//     (counted from 0), S_0 the state in front of it:
//       o_i = g^(i+1) S_0^T q_i + sum_(j<=i) g^(i-j) (q_i . k_j) v_j,    S_n = g^n S_0 + sum_j g^(n-1-j) k_j v_j^T
//     One kernel makes every chunk's own sum, one carries the state over the chunks (entry by entry, nothing but
//     S <- g^n S + U), one makes the outputs; chunks and heads are all parallel.  The powers of g come from a table.
#include "chunks.h"

namespace arle {

typedef float f32x4_t __attribute__((ext_vector_type(4)));

constexpr int kRetThreads = 256;
constexpr int kRetWaves = kRetThreads / kWave;

// ---- row by row ------------------------------------------------------------------------------------

// In place on float32 views: q and k turned, k scaled.
__global__ __launch_bounds__(kRetThreads) void retention_prep_kernel(float* __restrict__ q, long long q_stride,
                                                                     float* __restrict__ k, long long k_stride,
                                                                     const float* __restrict__ cos_t,
                                                                     const float* __restrict__ sin_t, int rot,
                                                                     const int* __restrict__ positions, int H, int D) {
  const int64_t t = blockIdx.x;
  const int half = rot / 2, per = D - half;   // a head's items: `half` pairs, then the entries that do not turn
  const int64_t angle = static_cast<int64_t>(positions[t]) * half;
  const float k_scale = 1.0f / sqrtf(static_cast<float>(D));
  float* qr = q + t * q_stride;
  float* kr = k + t * k_stride;
  for (int e = threadIdx.x; e < H * per; e += kRetThreads) {
    const int h = e / per, i = e % per;
    if (i < half) {
      const float c = cos_t[angle + i], s = sin_t[angle + i];
      float *qa = qr + h * D + i, *ka = kr + h * D + i;
      const float qu = qa[0], qv = qa[half], ku = ka[0], kv = ka[half];
      qa[0] = fmaf(qu, c, -qv * s);
      qa[half] = fmaf(qv, c, qu * s);
      ka[0] = fmaf(ku, c, -kv * s) * k_scale;
      ka[half] = fmaf(kv, c, ku * s) * k_scale;
    } else {
      kr[h * D + i + half] *= k_scale;
    }
  }
}

// A column of S never meets another: a workgroup a (request, head, 16 columns), four columns a wave, a sixteenth of D a
// lane; the sixteen shares of a column are the sixteen lanes of a row of the wave, which exchange by moves inside the
// vector unit.  Rows go through LDS in blocks of 32, fetched a block ahead.
constexpr int kScanCols = 16;
constexpr int kScanParts = 16;
constexpr int kScanRows = 32;
constexpr int kScanRowThreads = kRetThreads / kScanRows;

template <int CTRL>
__device__ __forceinline__ float lane_move(float v) {
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xf, 0xf, true));
}
// The sum over the sixteen lanes of a row, the same bits in each of them.
__device__ __forceinline__ float lanes16_sum(float v) {
  v += lane_move<0xB1>(v);    // quad_perm [1, 0, 3, 2]
  v += lane_move<0x4E>(v);    // quad_perm [2, 3, 0, 1]
  v += lane_move<0x141>(v);   // row_half_mirror
  v += lane_move<0x140>(v);   // row_mirror
  return v;
}

template <int DS>
__global__ __launch_bounds__(kRetThreads) void retention_scan_kernel(
    const float* __restrict__ q, long long q_stride, const float* __restrict__ k, long long k_stride,
    const float* __restrict__ v, long long v_stride, const float* __restrict__ decay, float* __restrict__ s_state,
    const int* __restrict__ seg_row0, const int* __restrict__ seg_slot, float* __restrict__ out /* [T, H * Dv] */, int H,
    int D, int Dv) {
  constexpr int DP = kScanParts * DS;   // padded D: what lies past D is zero
  constexpr int kMine = DP / kScanRowThreads, kValues = kScanRows * kScanCols / kRetThreads;
  __shared__ __attribute__((aligned(16))) float q_lds[kScanRows][DP];
  __shared__ __attribute__((aligned(16))) float k_lds[kScanRows][DP];
  __shared__ float v_lds[kScanRows][kScanCols];
  const int seg = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int lane = tid % kWave, wave = tid / kWave;
  const int col_in = wave * 4 + lane / kScanParts, col = blockIdx.z * kScanCols + col_in, part = lane % kScanParts;
  const bool live = col < Dv;
  const int row0 = seg_row0[seg], rows = seg_row0[seg + 1] - row0;
  float* s_ptr = s_state + (static_cast<int64_t>(seg_slot[seg]) * H + h) * D * Dv;
  const float g = decay[h];
  float S[DS];
#pragma unroll
  for (int i = 0; i < DS; ++i) {
    const int d = part * DS + i;
    S[i] = (live && d < D) ? s_ptr[static_cast<int64_t>(d) * Dv + col] : 0.f;
  }
  const int r = tid / kScanRowThreads, sub = tid % kScanRowThreads;
  float q_next[kMine], k_next[kMine], v_next[kValues];
  auto fetch = [&](int base) {
    const int n = min(kScanRows, rows - base);   // <= 0 behind the last block: nothing is loaded
    const int64_t t = row0 + base + min(r, max(n, 1) - 1);
#pragma unroll
    for (int j = 0; j < kMine; ++j) {
      const int d = sub + j * kScanRowThreads;
      const bool there = r < n && d < D;
      q_next[j] = there ? q[t * q_stride + h * D + d] : 0.f;
      k_next[j] = there ? k[t * k_stride + h * D + d] : 0.f;
    }
#pragma unroll
    for (int j = 0; j < kValues; ++j) {
      const int e = tid + j * kRetThreads, rr = e / kScanCols, c = blockIdx.z * kScanCols + e % kScanCols;
      v_next[j] = (rr < n && c < Dv) ? v[(row0 + base + rr) * v_stride + h * Dv + c] : 0.f;
    }
  };
  fetch(0);
  for (int base = 0; base < rows; base += kScanRows) {
    const int n = min(kScanRows, rows - base);
    __syncthreads();   // the block before has been read
#pragma unroll
    for (int j = 0; j < kMine; ++j) {
      q_lds[r][sub + j * kScanRowThreads] = q_next[j];
      k_lds[r][sub + j * kScanRowThreads] = k_next[j];
    }
#pragma unroll
    for (int j = 0; j < kValues; ++j) v_lds[(tid + j * kRetThreads) / kScanCols][(tid + j * kRetThreads) % kScanCols] = v_next[j];
    __syncthreads();
    fetch(base + kScanRows);
#pragma unroll 2
    for (int row = 0; row < n; ++row) {
      const float vv = v_lds[row][col_in];
      float sum[2] = {0.f, 0.f};
#pragma unroll
      for (int i = 0; i < DS; ++i) {
        S[i] = fmaf(k_lds[row][part * DS + i], vv, g * S[i]);
        sum[i % 2] = fmaf(S[i], q_lds[row][part * DS + i], sum[i % 2]);
      }
      const float o = lanes16_sum(sum[0] + sum[1]);
      if (part == 0 && live) out[static_cast<int64_t>(row0 + base + row) * (H * Dv) + h * Dv + col] = o;
    }
  }
#pragma unroll
  for (int i = 0; i < DS; ++i) {
    const int d = part * DS + i;
    if (live && d < D) s_ptr[static_cast<int64_t>(d) * Dv + col] = S[i];
  }
}

// One wave a (row, head).
__global__ __launch_bounds__(kWave) void retention_output_kernel(const float* __restrict__ o, const float* __restrict__ gate,
                                                                 long long gate_stride, float eps, void* __restrict__ out,
                                                                 int out_dtype, int H, int Dv) {
  const int64_t t = blockIdx.x;
  const int h = blockIdx.y, lane = threadIdx.x;
  const float* row = o + (t * H + h) * Dv;
  float ss = 0.f;
  for (int d = lane; d < Dv; d += kWave) ss = fmaf(row[d], row[d], ss);
  const float inv = 1.0f / sqrtf(wave_sum(ss) / static_cast<float>(Dv) + eps);
  for (int d = lane; d < Dv; d += kWave)
    store_from_float(out, out_dtype, (t * H + h) * Dv + d, row[d] * inv * gate_act(gate[t * gate_stride + h * Dv + d], kActSilu));
}

// ---- a decoded row ---------------------------------------------------------------------------------
// One workgroup a (request, head).  y: the fused product's sums, columns q | k | v | gate, as `parts` partial products
// that are added in order.  A thread holds four columns of S and walks rows d of it, RP rows a pass; Dv a multiple of 4
// up to 1024, D up to 256.
constexpr int kDecMaxD = 256, kDecMaxDv = 1024;
constexpr int kDecFlight = 8;   // rows of S a thread has in flight

__global__ __launch_bounds__(kRetThreads) void retention_decode_kernel(
    const float* __restrict__ y, int parts, long long part_stride, long long row_stride, const float* __restrict__ decay,
    const float* __restrict__ cos_t, const float* __restrict__ sin_t, int rot, const int* __restrict__ positions,
    const int* __restrict__ seg_row0, const int* __restrict__ seg_slot, float* __restrict__ s_state, float eps,
    void* __restrict__ out, int out_dtype, int H, int D, int Dv) {
  __shared__ float raw[2 * kDecMaxD];                                  // q, k as they came
  __shared__ float qk[2 * kDecMaxD];                                   // turned, k scaled
  __shared__ __attribute__((aligned(16))) float vs[kDecMaxDv];
  __shared__ __attribute__((aligned(16))) float os[4 * kRetThreads];   // partial read-outs, [pass row][Dv]
  __shared__ float red[kRetWaves];
  const int h = blockIdx.y, tid = threadIdx.x;
  const int64_t t = seg_row0[blockIdx.x];
  const int per_row = Dv / 4, RP = kRetThreads / per_row;              // threads a row of S, rows a pass
  const int rp = tid / per_row, c = 4 * (tid % per_row);
  const bool mine = rp < RP;
  float* s_ptr = s_state + (static_cast<int64_t>(seg_slot[blockIdx.x]) * H + h) * D * Dv;
  float4 next[kDecFlight];
  auto fetch = [&](int d0) {   // rows past D fetch the last row again and are dropped
#pragma unroll
    for (int u = 0; u < kDecFlight; ++u) next[u] = ld4<float>(s_ptr + static_cast<int64_t>(min(d0 + u * RP, D - 1)) * Dv + c);
  };
  fetch(min(rp, RP - 1));
  auto summed = [&](int64_t col) {
    const float* p = y + t * row_stride + col;
    float s = p[0];
    for (int i = 1; i < parts; ++i) s += p[i * part_stride];
    return s;
  };
  const int64_t qw = static_cast<int64_t>(H) * D, vw = static_cast<int64_t>(H) * Dv;
  for (int d = tid; d < 2 * D; d += kRetThreads) raw[d] = summed(d < D ? h * D + d : qw + h * D + d - D);
  for (int e = tid; e < Dv; e += kRetThreads) vs[e] = summed(2 * qw + h * Dv + e);
  __syncthreads();
  const int half = rot / 2;
  const int64_t angle = static_cast<int64_t>(positions[t]) * half;
  const float k_scale = 1.0f / sqrtf(static_cast<float>(D));
  for (int i = tid; i < 2 * D; i += kRetThreads) {
    const int d = i < D ? i : i - D, base = i - d;
    float x = raw[i];
    if (d < half)
      x = fmaf(x, cos_t[angle + d], -raw[base + d + half] * sin_t[angle + d]);
    else if (d < rot)
      x = fmaf(x, cos_t[angle + d - half], raw[base + d - half] * sin_t[angle + d - half]);
    qk[i] = base ? x * k_scale : x;
  }
  __syncthreads();
  const float g = decay[h];
  const float4 v4 = *reinterpret_cast<const float4*>(&vs[c]);
  float4 o = {0.f, 0.f, 0.f, 0.f};
  if (mine) {
    for (int d0 = rp; d0 < D; d0 += kDecFlight * RP) {
      float4 now[kDecFlight];
#pragma unroll
      for (int u = 0; u < kDecFlight; ++u) now[u] = next[u];
      if (d0 + kDecFlight * RP < D) fetch(d0 + kDecFlight * RP);
#pragma unroll
      for (int u = 0; u < kDecFlight; ++u) {
        const int d = d0 + u * RP;
        if (d < D) {
          const float kd = qk[D + d], qd = qk[d];
          float4 s = now[u];
          s.x = fmaf(kd, v4.x, g * s.x); s.y = fmaf(kd, v4.y, g * s.y);
          s.z = fmaf(kd, v4.z, g * s.z); s.w = fmaf(kd, v4.w, g * s.w);
          o.x = fmaf(qd, s.x, o.x); o.y = fmaf(qd, s.y, o.y); o.z = fmaf(qd, s.z, o.z); o.w = fmaf(qd, s.w, o.w);
          st4<float>(s_ptr + static_cast<int64_t>(d) * Dv + c, s);
        }
      }
    }
    *reinterpret_cast<float4*>(&os[rp * Dv + c]) = o;
  }
  __syncthreads();
  float ss = 0.f;
  for (int e = tid; e < Dv; e += kRetThreads) {
    float sum = 0.f;
    for (int p = 0; p < RP; ++p) sum += os[p * Dv + e];
    vs[e] = sum;      // (each thread its own entries: v has been read)
    ss = fmaf(sum, sum, ss);
  }
  const float inv = 1.0f / sqrtf(block_sum<kRetWaves>(ss, red) / static_cast<float>(Dv) + eps);
  for (int e = tid; e < Dv; e += kRetThreads)
    store_from_float(out, out_dtype, (t * H + h) * Dv + e, vs[e] * inv * gate_act(summed(2 * qw + vw + h * Dv + e), kActSilu));
}

// ---- chunks of rows on the matrix cores ------------------------------------------------------------
// v_mfma_f32_16x16x4_f32: a lane gives A[i = lane % 16][k = lane / 16] and B[k][j = lane % 16]; the result's lane holds
// rows 4 (lane / 16) .. + 3 of column lane % 16.  Operands that lie along k are read four at a time: the four products
// of sixteen k take k = 4 g + j, j = 0..3, g = lane / 16, the same for both operands.
constexpr int kChunk = kChunkRows;
constexpr int kSliceD = 64, kSliceRow = kSliceD + 4;    // a slice of q and k in LDS, a row padded by four

__device__ __forceinline__ f32x4_t mfma4(const float4& a, const float4& b, f32x4_t acc) {
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b.x, acc, 0, 0, 0);
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b.y, acc, 0, 0, 0);
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b.z, acc, 0, 0, 0);
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b.w, acc, 0, 0, 0);
}

// Four entries d .. d + 3 of a row x of D entries turned by the angles at `cs`, `sn` (half entries a position).  The loads
// stand under no condition: entries that do not turn fetch an angle and drop it.
__device__ __forceinline__ float4 turned4(const float* x, int d, int rot, const float* cs, const float* sn) {
  const float4 v = ld4<float>(x + d);
  if (rot == 0) return v;
  const int half = rot / 2;
  const bool turns = d < rot, first = d < half;
  const int a = turns ? (first ? d : d - half) : 0;
  const float4 o = ld4<float>(x + (turns ? (first ? d + half : d - half) : d)), c = ld4<float>(cs + a), s = ld4<float>(sn + a);
  const float sign = first ? -1.f : 1.f;
  const float4 t = {fmaf(v.x, c.x, sign * o.x * s.x), fmaf(v.y, c.y, sign * o.y * s.y), fmaf(v.z, c.z, sign * o.z * s.z), fmaf(v.w, c.w, sign * o.w * s.w)};
  return turns ? t : v;
}

struct ChunkArgs {
  const float* y;           // [T, .]: columns q | k | v | gate
  long long row_stride;
  const float* cos_t;
  const float* sin_t;
  int rot;
  const int* positions;
  const int* seg_row0;
  const int* seg_slot;
  int segments;
  const float* powers;      // [H, 65]: g_h^0 .. g_h^64
  float* s_state;
  float* work;              // [items, H, Dv, D]: a chunk's own sum, then the state in front of it (transposed)
  int H, D, Dv;
};

// U^T of a chunk: work[item, h, e, d] = sum_j g^(n-1-j) k_j[d] v_j[e].
// NE: tiles of sixteen columns a wave takes at a time; the columns are padded with zeros to whole groups of them.
template <int NE>
__global__ __launch_bounds__(kRetThreads) void retention_chunk_sum_kernel(const ChunkArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const ChunkAt at = find_chunk(a.seg_row0, a.segments, blockIdx.x);
  if (at.rows == 0) return;
  const int h = blockIdx.y, tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, n = lane % 16, g = lane / 16;
  const int D = a.D, Dv = a.Dv, DP = (D + 15) / 16 * 16, EP = (Dv + 16 * NE - 1) / (16 * NE) * 16 * NE, kr = DP + 4, vr = EP + 4;
  float* ks = lds;                      // [64][DP + 4]
  float* vs = lds + kChunk * kr;        // [64][EP + 4]
  const int64_t qw = static_cast<int64_t>(a.H) * D;
  const float* pw = a.powers + h * (kChunk + 1);
  const float k_scale = 1.0f / sqrtf(static_cast<float>(D));
  const int steps = (at.rows + 15) / 16;      // sixteen rows at a time; rows past the chunk's are zero
  // Staged four pieces a thread at a time, their loads in flight together: a piece past the chunk's rows or past a row's
  // entries fetches one inside and becomes zero.
  const int64_t pos0 = a.positions[at.row0];      // a segment's positions follow one another
  const float* y0 = a.y + at.row0 * a.row_stride + qw;
  for (int base = 0; base < steps * 16 * (DP / 4); base += 4 * kRetThreads) {
    float4 v[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int i = base + u * kRetThreads + tid, r = min(i / (DP / 4), at.rows - 1), d = min(4 * (i % (DP / 4)), D - 4);
      const int64_t ang = (pos0 + r) * (a.rot / 2);
      v[u] = turned4(y0 + r * a.row_stride + h * D, d, a.rot, a.cos_t + ang, a.sin_t + ang);
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int i = base + u * kRetThreads + tid, r = i / (DP / 4), d = 4 * (i % (DP / 4));
      const float f = (r < at.rows && d < D) ? k_scale * pw[max(at.rows - 1 - r, 0)] : 0.f;
      if (i < steps * 16 * (DP / 4)) *reinterpret_cast<float4*>(&ks[r * kr + d]) = float4{v[u].x * f, v[u].y * f, v[u].z * f, v[u].w * f};
    }
  }
  for (int base = 0; base < steps * 16 * (EP / 4); base += 4 * kRetThreads) {
    float4 v[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int i = base + u * kRetThreads + tid, r = min(i / (EP / 4), at.rows - 1), e = min(4 * (i % (EP / 4)), Dv - 4);
      v[u] = ld4<float>(y0 + r * a.row_stride + qw + h * Dv + e);
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int i = base + u * kRetThreads + tid, r = i / (EP / 4), e = 4 * (i % (EP / 4));
      if (i < steps * 16 * (EP / 4))
        *reinterpret_cast<float4*>(&vs[r * vr + e]) = (r < at.rows && e < Dv) ? v[u] : float4{0.f, 0.f, 0.f, 0.f};
    }
  }
  __syncthreads();
  float* dst = a.work + (static_cast<int64_t>(blockIdx.x) * a.H + h) * D * Dv;
  for (int d0 = 16 * wave; d0 < DP; d0 += 16 * kRetWaves) {
    for (int e0 = 0; e0 < EP; e0 += 16 * NE) {
      f32x4_t acc[NE];
#pragma unroll
      for (int j = 0; j < NE; ++j) acc[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
      for (int s = 0; s < steps; ++s) {
        const int r = 16 * s + 4 * g;
        const float* kp = ks + r * kr + d0 + n;
        const float4 ka = {kp[0], kp[kr], kp[2 * kr], kp[3 * kr]};
#pragma unroll
        for (int j = 0; j < NE; ++j) {
          const float* vp = vs + r * vr + e0 + 16 * j + n;
          acc[j] = mfma4(ka, float4{vp[0], vp[vr], vp[2 * vr], vp[3 * vr]}, acc[j]);
        }
      }
#pragma unroll
      for (int j = 0; j < NE; ++j) {
        const int e = e0 + 16 * j + n, d = d0 + 4 * g;
        if (e < Dv && d < D) st4<float>(dst + static_cast<int64_t>(e) * D + d, float4{acc[j][0], acc[j][1], acc[j][2], acc[j][3]});
      }
    }
  }
}

// The state carried over a request's chunks: work becomes the state in front of each chunk, s_state the one behind the
// last.  A thread takes four entries d .. d + 3 of one column e.
constexpr int kCarryFlight = 8;

__global__ __launch_bounds__(kRetThreads) void retention_chunk_carry_kernel(const ChunkArgs a) {
  const int seg = blockIdx.x, h = blockIdx.y, D = a.D, Dv = a.Dv;
  const int i = blockIdx.z * kRetThreads + threadIdx.x;
  if (i >= D / 4 * Dv) return;
  const int e = i / (D / 4), d = 4 * (i % (D / 4));
  int first = 0;
  for (int s = 0; s < seg; ++s) first += (a.seg_row0[s + 1] - a.seg_row0[s] + kChunk - 1) / kChunk;
  const int rows = a.seg_row0[seg + 1] - a.seg_row0[seg], chunks = (rows + kChunk - 1) / kChunk;
  if (chunks == 0) return;
  float* st = a.s_state + (static_cast<int64_t>(a.seg_slot[seg]) * a.H + h) * D * Dv + static_cast<int64_t>(d) * Dv + e;
  float4 S = {st[0], st[Dv], st[2 * Dv], st[3 * Dv]};
  const int64_t step = static_cast<int64_t>(a.H) * D * Dv;
  float* w = a.work + (static_cast<int64_t>(first) * a.H + h) * D * Dv + static_cast<int64_t>(e) * D + d;
  const float* pw = a.powers + h * (kChunk + 1);
  const float full = pw[kChunk], part = pw[rows - (chunks - 1) * kChunk];
  for (int c0 = 0; c0 < chunks; c0 += kCarryFlight) {
    float4 u[kCarryFlight];
#pragma unroll
    for (int j = 0; j < kCarryFlight; ++j) u[j] = ld4<float>(w + min(c0 + j, chunks - 1) * step);
#pragma unroll
    for (int j = 0; j < kCarryFlight; ++j) {
      if (c0 + j < chunks) {
        st4<float>(w + (c0 + j) * step, S);
        const float f = c0 + j == chunks - 1 ? part : full;
        S = float4{fmaf(f, S.x, u[j].x), fmaf(f, S.y, u[j].y), fmaf(f, S.z, u[j].z), fmaf(f, S.w, u[j].w)};
      }
    }
  }
  st[0] = S.x; st[Dv] = S.y; st[2 * Dv] = S.z; st[3 * Dv] = S.w;
}

// The outputs of a chunk: wave w makes rows 16 w .. + 15 in all columns, norms them and applies the gate.
template <int NV>
__global__ __launch_bounds__(kRetThreads) void retention_chunk_out_kernel(const ChunkArgs a, float eps, void* __restrict__ out,
                                                                          int out_dtype) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float pw[kChunk + 1];
  const ChunkAt at = find_chunk(a.seg_row0, a.segments, blockIdx.x);
  if (at.rows == 0) return;
  const int h = blockIdx.y, tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, n = lane % 16, g = lane / 16;
  const int D = a.D, Dv = a.Dv;
  constexpr int EP = 16 * NV, vr = EP + 4;         // columns, those past Dv zero
  float* qs = lds;                                 // [64][68] q's slice, then k's; later v, [64][EP + 4]
  float* ks = qs + kChunk * kSliceRow;
  float* vs = qs;
  float* ss = lds + kChunk * max(2 * kSliceRow, vr);   // [EP][68] the state's slice; later the masked scores, [64][68]
  float* ps = ss;
  const int64_t qw = static_cast<int64_t>(a.H) * D;
  const float k_scale = 1.0f / sqrtf(static_cast<float>(D));
  if (tid <= kChunk) pw[tid] = a.powers[h * (kChunk + 1) + tid];
  const int64_t pos0 = a.positions[at.row0];       // a segment's positions follow one another
  const float* S0 = a.work + (static_cast<int64_t>(blockIdx.x) * a.H + h) * D * Dv;     // [e][d]
  const int blocks = (at.rows + 15) / 16;          // row blocks of sixteen that hold rows
  const float4 zero = {0.f, 0.f, 0.f, 0.f};
  f32x4_t p[4], o[NV];
#pragma unroll
  for (int j = 0; j < 4; ++j) p[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int j = 0; j < NV; ++j) o[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float4 v_next[NV];                               // the chunk's values, 64 rows of EP entries over the workgroup
#pragma unroll
  for (int x = 0; x < NV; ++x) {
    const int i = x * kRetThreads + tid, r = min(i / (EP / 4), at.rows - 1), e = min(4 * (i % (EP / 4)), Dv - 4);
    v_next[x] = ld4<float>(a.y + (at.row0 + r) * a.row_stride + 2 * qw + h * Dv + e);
  }
  for (int d0 = 0; d0 < D; d0 += kSliceD) {
    float4 s_next[NV];                             // EP rows of 64 over the workgroup
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const int i = x * kRetThreads + tid, e = min(i / (kSliceD / 4), Dv - 1), d = min(d0 + 4 * (i % (kSliceD / 4)), D - 4);
      s_next[x] = ld4<float>(S0 + static_cast<int64_t>(e) * D + d);
    }
    __syncthreads();                               // the slice before has been read
#pragma unroll 2
    for (int x = 0; x < kChunk * (kSliceD / 4) / kRetThreads; ++x) {
      const int i = x * kRetThreads + tid, r = i / (kSliceD / 4), c = 4 * (i % (kSliceD / 4)), rr = min(r, at.rows - 1);
      const int d = min(d0 + c, D - 4);
      const bool in = r < at.rows && d0 + c < D;
      const int64_t ang = (pos0 + rr) * (a.rot / 2);
      const float* row = a.y + (at.row0 + rr) * a.row_stride + h * D;
      const float4 q4 = turned4(row, d, a.rot, a.cos_t + ang, a.sin_t + ang), k4 = turned4(row + qw, d, a.rot, a.cos_t + ang, a.sin_t + ang);
      *reinterpret_cast<float4*>(&qs[r * kSliceRow + c]) = in ? q4 : zero;
      *reinterpret_cast<float4*>(&ks[r * kSliceRow + c]) =
          in ? float4{k4.x * k_scale, k4.y * k_scale, k4.z * k_scale, k4.w * k_scale} : zero;
    }
#pragma unroll
    for (int x = 0; x < NV; ++x) {                 // (past D the query's slice is zero, columns past Dv are dropped)
      const int i = x * kRetThreads + tid;
      *reinterpret_cast<float4*>(&ss[(i / (kSliceD / 4)) * kSliceRow + 4 * (i % (kSliceD / 4))]) = s_next[x];
    }
    __syncthreads();
    if (wave < blocks) {
#pragma unroll
      for (int kk = 0; kk < kSliceD; kk += 16) {   // (past D the slices of q and k are zero)
        const int c = kk + 4 * g;
        const float4 qa = *reinterpret_cast<const float4*>(&qs[(16 * wave + n) * kSliceRow + c]);
#pragma unroll
        for (int j = 0; j < 4; ++j) p[j] = mfma4(qa, *reinterpret_cast<const float4*>(&ks[(16 * j + n) * kSliceRow + c]), p[j]);
#pragma unroll
        for (int j = 0; j < NV; ++j) o[j] = mfma4(qa, *reinterpret_cast<const float4*>(&ss[(16 * j + n) * kSliceRow + c]), o[j]);
      }
    }
  }
  __syncthreads();                                 // the last slices have been read by every wave
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = 16 * wave + 4 * g + i;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = 16 * j + n;
      ps[r * kSliceRow + c] = c <= r ? p[j][i] * pw[r - c] : 0.f;
    }
#pragma unroll
    for (int j = 0; j < NV; ++j) o[j][i] *= pw[r + 1];
  }
  // the gates are asked for now, in front of the last products (rows and columns past the end: one inside, dropped)
  float gates[4][NV];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int64_t t = at.row0 + min(16 * wave + 4 * g + i, at.rows - 1);
    const float* gate = a.y + t * a.row_stride + 2 * qw + static_cast<int64_t>(a.H) * Dv + h * Dv;
#pragma unroll
    for (int j = 0; j < NV; ++j) gates[i][j] = gate[min(16 * j + n, Dv - 1)];
  }
#pragma unroll
  for (int x = 0; x < NV; ++x) {
    const int i = x * kRetThreads + tid, r = i / (EP / 4), e = 4 * (i % (EP / 4));
    *reinterpret_cast<float4*>(&vs[r * vr + e]) = (r < at.rows && e < Dv) ? v_next[x] : zero;
  }
  __syncthreads();
  if (wave >= blocks) return;
  for (int s = 0; s <= wave; ++s) {                // (a wave's own rows: what it wrote of ps it reads itself)
    const int r = 16 * s + 4 * g;
    const float4 pa = *reinterpret_cast<const float4*>(&ps[(16 * wave + n) * kSliceRow + r]);
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const float* vp = vs + r * vr + 16 * j + n;
      o[j] = mfma4(pa, float4{vp[0], vp[vr], vp[2 * vr], vp[3 * vr]}, o[j]);
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = 16 * wave + 4 * g + i;
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < NV; ++j)
      if (16 * j + n < Dv) ss = fmaf(o[j][i], o[j][i], ss);
    const float inv = 1.0f / sqrtf(lanes16_sum(ss) / static_cast<float>(Dv) + eps);
    if (r >= at.rows) continue;
    const int64_t t = at.row0 + r;
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int e = 16 * j + n;
      if (e < Dv) store_from_float(out, out_dtype, (t * a.H + h) * Dv + e, o[j][i] * inv * gate_act(gates[i][j], kActSilu));
    }
  }
}

}  // namespace arle

using namespace arle;

// q, k: float32 [T, H * D] views, in place.  cos, sin: float32 [positions, rot / 2].
extern "C" int arle_retention_prep(float* q, long long q_stride, float* k, long long k_stride, const float* cos_t,
                                   const float* sin_t, int rot, const int* positions, int tokens, int H, int D, void* stream) {
  if (tokens == 0) return 0;
  if (H < 1 || D < 1 || rot < 0 || rot > D || rot % 2 || (rot && (!cos_t || !sin_t))) return static_cast<int>(hipErrorInvalidValue);
  retention_prep_kernel<<<tokens, kRetThreads, 0, static_cast<hipStream_t>(stream)>>>(q, q_stride, k, k_stride, cos_t, sin_t,
                                                                                      rot, positions, H, D);
  return launch_status();
}

// q, k (prepared) [T, H * D], v [T, H * Dv]: float32 views; out float32 [T, H * Dv] contiguous.
extern "C" int arle_retention_scan(const float* q, long long q_stride, const float* k, long long k_stride, const float* v,
                                   long long v_stride, const float* decay, float* s_state, const int* seg_row0,
                                   const int* seg_slot, int segments, float* out, int H, int D, int Dv, void* stream) {
  if (segments == 0) return 0;
  if (H < 1 || H > 65535 || D < 1 || D > 256 || Dv < 1) return static_cast<int>(hipErrorInvalidValue);
  const dim3 grid(segments, H, (Dv + kScanCols - 1) / kScanCols);
  hipStream_t s = static_cast<hipStream_t>(stream);
#define ARLE_RS(DS)                                                                                                     \
  retention_scan_kernel<DS><<<grid, kRetThreads, 0, s>>>(q, q_stride, k, k_stride, v, v_stride, decay, s_state, seg_row0, \
                                                         seg_slot, out, H, D, Dv)
  if (D <= 32) ARLE_RS(2); else if (D <= 64) ARLE_RS(4); else if (D <= 128) ARLE_RS(8); else ARLE_RS(16);
#undef ARLE_RS
  return launch_status();
}

extern "C" int arle_retention_output(const float* o, const float* gate, long long gate_stride, float eps, void* out,
                                     int out_dtype, int tokens, int H, int Dv, void* stream) {
  if (tokens == 0) return 0;
  if (H < 1 || H > 65535 || Dv < 1) return static_cast<int>(hipErrorInvalidValue);
  retention_output_kernel<<<dim3(tokens, H), kWave, 0, static_cast<hipStream_t>(stream)>>>(o, gate, gate_stride, eps, out,
                                                                                           out_dtype, H, Dv);
  return launch_status();
}

// y float32: `parts` partial products part_stride apart of rows row_stride apart, columns q | k | v | gate; one row a
// segment.  out [T, H * Dv] of out_dtype.
extern "C" int arle_retention_decode(const float* y, int parts, long long part_stride, long long row_stride,
                                     const float* decay, const float* cos_t, const float* sin_t, int rot,
                                     const int* positions, const int* seg_row0, const int* seg_slot, float* s_state,
                                     float eps, void* out, int out_dtype, int segments, int H, int D, int Dv, void* stream) {
  if (segments == 0) return 0;
  if (parts < 1 || H < 1 || H > 65535 || D < 1 || D > kDecMaxD || Dv < 4 || Dv > kDecMaxDv || Dv % 4 || rot < 0 || rot > D ||
      rot % 2 || (rot && (!cos_t || !sin_t)) || reinterpret_cast<uintptr_t>(s_state) % 16)
    return static_cast<int>(hipErrorInvalidValue);
  retention_decode_kernel<<<dim3(segments, H), kRetThreads, 0, static_cast<hipStream_t>(stream)>>>(
      y, parts, part_stride, row_stride, decay, cos_t, sin_t, rot, positions, seg_row0, seg_slot, s_state, eps, out,
      out_dtype, H, D, Dv);
  return launch_status();
}

// y float32 [T, .], columns q | k | v | gate.  powers float32 [H, 65].  work: float32 [items, H, Dv, D] with items at
// least the number of chunks of 64 rows of all segments.  out [T, H * Dv] of out_dtype.
extern "C" int arle_retention_chunks(const float* y, long long row_stride, const float* cos_t, const float* sin_t, int rot,
                                     const int* positions, const int* seg_row0, const int* seg_slot, const float* powers,
                                     float* s_state, int segments, int items, float* work, float eps, void* out,
                                     int out_dtype, int H, int D, int Dv, void* stream) {
  if (segments == 0 || items == 0) return 0;
  auto al = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  if (H < 1 || H > 65535 || D < 4 || D > 256 || D % 4 || Dv < 4 || Dv > 256 || Dv % 4 || rot < 0 || rot > D || rot % 8 ||
      (rot && (!cos_t || !sin_t || !al(cos_t) || !al(sin_t))) || row_stride % 4 || !al(y) || !al(work))
    return static_cast<int>(hipErrorInvalidValue);
  const ChunkArgs a{y, row_stride, cos_t, sin_t, rot, positions, seg_row0, seg_slot, segments, powers, s_state, work, H, D, Dv};
  hipStream_t s = static_cast<hipStream_t>(stream);
  const int DP = (D + 15) / 16 * 16;
  const int columns = Dv <= 64 ? 64 : (Dv <= 128 ? 128 : 256);
  const size_t sum_lds = static_cast<size_t>(kChunk) * (DP + 4 + columns + 4) * sizeof(float);
  const size_t out_lds = (static_cast<size_t>(kChunk) * max(2 * kSliceRow, columns + 4) + static_cast<size_t>(columns) * kSliceRow) * sizeof(float);
  static bool raised = false;
  if (!raised) {
    const void* kernels[] = {reinterpret_cast<const void*>(&retention_chunk_sum_kernel<4>),
                             reinterpret_cast<const void*>(&retention_chunk_sum_kernel<8>),
                             reinterpret_cast<const void*>(&retention_chunk_out_kernel<4>),
                             reinterpret_cast<const void*>(&retention_chunk_out_kernel<8>),
                             reinterpret_cast<const void*>(&retention_chunk_out_kernel<16>)};
    for (const void* f : kernels) {
      const hipError_t e = hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, 144 * 1024);
      if (e != hipSuccess) return static_cast<int>(e);
    }
    raised = true;
  }
  const dim3 grid(items, H);
  if (columns == 64)
    retention_chunk_sum_kernel<4><<<grid, kRetThreads, sum_lds, s>>>(a);
  else
    retention_chunk_sum_kernel<8><<<grid, kRetThreads, sum_lds, s>>>(a);
  retention_chunk_carry_kernel<<<dim3(segments, H, (D / 4 * Dv + kRetThreads - 1) / kRetThreads), kRetThreads, 0, s>>>(a);
  if (columns == 64)
    retention_chunk_out_kernel<4><<<grid, kRetThreads, out_lds, s>>>(a, eps, out, out_dtype);
  else if (columns == 128)
    retention_chunk_out_kernel<8><<<grid, kRetThreads, out_lds, s>>>(a, eps, out, out_dtype);
  else
    retention_chunk_out_kernel<16><<<grid, kRetThreads, out_lds, s>>>(a, eps, out, out_dtype);
  return launch_status();
}
