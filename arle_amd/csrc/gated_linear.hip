// Gated linear attention for the rows of a packed step, continued across steps through a per-request state
// S [heads, D, Dv] in 32-bit floats: a decay for every head and key entry, made from the token.
//
//   S_t = diag(a_t) S_(t-1) + k_t v_t^T,   o_t = D^(-1/2) S_t^T q_t,   y_t = o_t / sqrt(mean(o_t^2) + eps) * w * silu(gate_t)
//   a = sigmoid(W m + b)^(1/tau), m the narrow middle of two projections
//
// All in 32-bit arithmetic from the projections' 32-bit sums on (columns q | k | v | gate | middle of one product).  Two forms
// beside the one row by row in decay_scan.hip:
//   * a decoded row (`gated_linear_decode`): one kernel from the product's partial sums to y;
//   * chunks of 64 rows on the matrix cores' float32 products.  With B_i[d] the sum of log a over the chunk's rows up to i
//     (made by `decay_gates`), S_0 the state in front of a chunk of n rows:
//       o_i = S_0^T (q_i exp(B_i)) + sum_(j<=i) P_ij v_j,    P_ij = sum_d q_i[d] k_j[d] exp(B_i[d] - B_j[d])
//       S_n = diag(exp(B_(n-1))) S_0 + sum_j (k_j exp(B_(n-1) - B_j)) v_j^T
//     One kernel makes every chunk's own sum, one carries the state over the chunks, one makes the outputs.
// The exponential in P stands between two rows and a key entry; a matrix product needs it in two factors.  Rows go in blocks
// of sixteen.  With E_J the sum B behind the last row of block J, k counts exp(E_J - B_j) (at most 1, once for all queries),
// and q counts exp(B_i - E_J): at most 1 for blocks in front of the query's own.  For the own block that factor grows with
// what the block forgets; where it would pass exp(40) (decays close to 0), that block's P is made pair by pair instead.
#include "chunks.h"
#include "lane_sums.h"

namespace arle {

typedef float f32x4_t __attribute__((ext_vector_type(4)));

constexpr int kGlThreads = 256;
constexpr int kGlWaves = kGlThreads / kWave;

// ---- a decoded row ---------------------------------------------------------------------------------
// One workgroup a (request, head).  A thread holds four columns of S and walks rows d of it, RP rows a pass; Dv a multiple of 4
// up to 1024, D and the middle up to 256.
constexpr int kGlMaxD = 256, kGlMaxDv = 1024, kGlMaxRank = 256;
constexpr int kGlFlight = 8;   // rows of S a thread has in flight

template <typename TW>
__global__ __launch_bounds__(kGlThreads) void gated_linear_decode_kernel(
    const float* __restrict__ y, int parts, long long part_stride, long long row_stride, const TW* __restrict__ a2, int rank,
    const float* __restrict__ a2_bias, float inv_tau, const float* __restrict__ norm, const int* __restrict__ seg_row0,
    const int* __restrict__ seg_slot, float* __restrict__ s_state, float eps, void* __restrict__ out, int out_dtype, int H, int D,
    int Dv) {
  __shared__ float qk[2 * kGlMaxD];                                   // q scaled, k
  __shared__ float decay[kGlMaxD];
  __shared__ float mid[kGlMaxRank];
  __shared__ __attribute__((aligned(16))) float vs[kGlMaxDv];
  __shared__ float gs[kGlMaxDv];
  __shared__ __attribute__((aligned(16))) float os[4 * kGlThreads];   // partial read-outs, [pass row][Dv]
  __shared__ float red[kGlWaves];
  const int h = blockIdx.y, tid = threadIdx.x;
  const int64_t t = seg_row0[blockIdx.x];
  const int per_row = Dv / 4, RP = kGlThreads / per_row;              // threads a row of S, rows a pass
  const int rp = tid / per_row, c = 4 * (tid % per_row);
  const bool mine = rp < RP;
  float* s_ptr = s_state + (static_cast<int64_t>(seg_slot[blockIdx.x]) * H + h) * D * Dv;
  float4 next[kGlFlight];
  auto fetch = [&](int d0) {   // rows past D fetch the last row again and are dropped
#pragma unroll
    for (int u = 0; u < kGlFlight; ++u) next[u] = ld4<float>(s_ptr + static_cast<int64_t>(min(d0 + u * RP, D - 1)) * Dv + c);
  };
  fetch(min(rp, RP - 1));
  const int64_t qw = static_cast<int64_t>(H) * D, vw = static_cast<int64_t>(H) * Dv;
  const float* yr = y + t * row_stride;
  for (int r = tid; r < rank; r += kGlThreads) mid[r] = sum_parts(yr + 2 * qw + 2 * vw + r, parts, part_stride);
  const float q_scale = 1.0f / sqrtf(static_cast<float>(D));
  for (int d = tid; d < 2 * D; d += kGlThreads) {
    const float x = sum_parts(yr + (d < D ? h * D + d : qw + h * D + d - D), parts, part_stride);
    qk[d] = d < D ? x * q_scale : x;
  }
  for (int e = tid; e < Dv; e += kGlThreads) {
    vs[e] = sum_parts(yr + 2 * qw + h * Dv + e, parts, part_stride);
    gs[e] = sum_parts(yr + 2 * qw + vw + h * Dv + e, parts, part_stride);
  }
  __syncthreads();
  for (int d = tid; d < D; d += kGlThreads) {
    const TW* w = a2 + static_cast<int64_t>(h * D + d) * rank;
    float z = 0.f;
#pragma unroll 8
    for (int r = 0; r < rank; ++r) z = fmaf(to_float(w[r]), mid[r], z);
    decay[d] = expf(-softplus_f(-(z + a2_bias[h * D + d])) * inv_tau);
  }
  __syncthreads();
  const float4 v4 = *reinterpret_cast<const float4*>(&vs[c]);
  float4 o = {0.f, 0.f, 0.f, 0.f};
  if (mine) {
    for (int d0 = rp; d0 < D; d0 += kGlFlight * RP) {
      float4 now[kGlFlight];
#pragma unroll
      for (int u = 0; u < kGlFlight; ++u) now[u] = next[u];
      if (d0 + kGlFlight * RP < D) fetch(d0 + kGlFlight * RP);
#pragma unroll
      for (int u = 0; u < kGlFlight; ++u) {
        const int d = d0 + u * RP;
        if (d < D) {
          const float kd = qk[D + d], qd = qk[d], g = decay[d];
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
  for (int e = tid; e < Dv; e += kGlThreads) {
    float sum = 0.f;
    for (int p = 0; p < RP; ++p) sum += os[p * Dv + e];
    vs[e] = sum;      // (each thread its own entries: v has been read)
    ss = fmaf(sum, sum, ss);
  }
  const float inv = 1.0f / sqrtf(block_sum<kGlWaves>(ss, red) / static_cast<float>(Dv) + eps);
  for (int e = tid; e < Dv; e += kGlThreads)
    store_from_float(out, out_dtype, (t * H + h) * Dv + e, vs[e] * inv * norm[e] * gate_act(gs[e], kActSilu));
}

// ---- chunks of rows on the matrix cores ------------------------------------------------------------
// v_mfma_f32_16x16x4_f32: a lane gives A[i = lane % 16][k = lane / 16] and B[k][j = lane % 16]; the result's lane holds
// rows 4 (lane / 16) .. + 3 of column lane % 16.  Operands that lie along k are read four at a time: the four products
// of sixteen k take k = 4 g + j, j = 0..3, g = lane / 16, the same for both operands.
constexpr int kGlSlice = 64, kGlSliceRow = kGlSlice + 4;    // a slice of D in LDS, a row padded by four
constexpr float kGlMaxGrowth = 40.f;                        // exponent up to which a query's factor stays a factor

__device__ __forceinline__ f32x4_t mfma4(const float4& a, const float4& b, f32x4_t acc) {
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b.x, acc, 0, 0, 0);
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b.y, acc, 0, 0, 0);
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b.z, acc, 0, 0, 0);
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b.w, acc, 0, 0, 0);
}

__device__ __forceinline__ float4 times_exp(const float4& x, const float4& b, const float4& from) {   // x exp(b - from)
  return float4{x.x * __expf(b.x - from.x), x.y * __expf(b.y - from.y), x.z * __expf(b.z - from.z), x.w * __expf(b.w - from.w)};
}

struct GlChunkArgs {
  const float* y;           // [T, .]: columns q | k | v | gate
  long long row_stride;
  const float* sums;        // [T, H * D]: B, the logarithms of the decays summed up from the chunk's first row on
  const int* seg_row0;
  const int* seg_slot;
  int segments;
  float* s_state;
  float* work;              // [items, H, Dv, D]: a chunk's own sum, then the state in front of it (transposed)
  int H, D, Dv;
};

// U^T of a chunk: work[item, h, e, d] = sum_j k_j[d] exp(B_(n-1)[d] - B_j[d]) v_j[e].
// NE: tiles of sixteen columns a wave takes at a time; the columns are padded with zeros to whole groups of them.
template <int NE>
__global__ __launch_bounds__(kGlThreads) void gated_linear_chunk_sum_kernel(const GlChunkArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const ChunkAt at = find_chunk(a.seg_row0, a.segments, blockIdx.x);
  if (at.rows == 0) return;
  const int h = blockIdx.y, tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, n = lane % 16, g = lane / 16;
  const int D = a.D, Dv = a.Dv, DP = (D + 15) / 16 * 16, EP = (Dv + 16 * NE - 1) / (16 * NE) * 16 * NE, kr = DP + 4, vr = EP + 4;
  float* ks = lds;                           // [64][DP + 4]
  float* vs = lds + kChunkRows * kr;         // [64][EP + 4]
  const int64_t qw = static_cast<int64_t>(a.H) * D;
  const int steps = (at.rows + 15) / 16;     // sixteen rows at a time; rows past the chunk's are zero
  // Staged four pieces a thread at a time, their loads in flight together: a piece past the chunk's rows or past a row's
  // entries fetches one inside and becomes zero.
  const float* y0 = a.y + at.row0 * a.row_stride + qw;
  const float* b0 = a.sums + at.row0 * qw + h * D;
  for (int base = 0; base < steps * 16 * (DP / 4); base += 4 * kGlThreads) {
    float4 v[4], b[4], end[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int i = base + u * kGlThreads + tid, r = min(i / (DP / 4), at.rows - 1), d = min(4 * (i % (DP / 4)), D - 4);
      v[u] = ld4<float>(y0 + r * a.row_stride + h * D + d);
      b[u] = ld4<float>(b0 + r * qw + d);
      end[u] = ld4<float>(b0 + (at.rows - 1) * qw + d);
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int i = base + u * kGlThreads + tid, r = i / (DP / 4), d = 4 * (i % (DP / 4));
      const bool in = r < at.rows && d < D;
      if (i < steps * 16 * (DP / 4))
        *reinterpret_cast<float4*>(&ks[r * kr + d]) = in ? times_exp(v[u], end[u], b[u]) : float4{0.f, 0.f, 0.f, 0.f};
    }
  }
  for (int base = 0; base < steps * 16 * (EP / 4); base += 4 * kGlThreads) {
    float4 v[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int i = base + u * kGlThreads + tid, r = min(i / (EP / 4), at.rows - 1), e = min(4 * (i % (EP / 4)), Dv - 4);
      v[u] = ld4<float>(y0 + r * a.row_stride + qw + h * Dv + e);
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int i = base + u * kGlThreads + tid, r = i / (EP / 4), e = 4 * (i % (EP / 4));
      if (i < steps * 16 * (EP / 4))
        *reinterpret_cast<float4*>(&vs[r * vr + e]) = (r < at.rows && e < Dv) ? v[u] : float4{0.f, 0.f, 0.f, 0.f};
    }
  }
  __syncthreads();
  float* dst = a.work + (static_cast<int64_t>(blockIdx.x) * a.H + h) * D * Dv;
  for (int d0 = 16 * wave; d0 < DP; d0 += 16 * kGlWaves) {
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
constexpr int kGlCarryFlight = 8;

__global__ __launch_bounds__(kGlThreads) void gated_linear_chunk_carry_kernel(const GlChunkArgs a) {
  const int seg = blockIdx.x, h = blockIdx.y, D = a.D, Dv = a.Dv;
  const int i = blockIdx.z * kGlThreads + threadIdx.x;
  if (i >= D / 4 * Dv) return;
  const int e = i / (D / 4), d = 4 * (i % (D / 4));
  int first = 0;
  for (int s = 0; s < seg; ++s) first += (a.seg_row0[s + 1] - a.seg_row0[s] + kChunkRows - 1) / kChunkRows;
  const int row0 = a.seg_row0[seg], rows = a.seg_row0[seg + 1] - row0, chunks = (rows + kChunkRows - 1) / kChunkRows;
  if (chunks == 0) return;
  float* st = a.s_state + (static_cast<int64_t>(a.seg_slot[seg]) * a.H + h) * D * Dv + static_cast<int64_t>(d) * Dv + e;
  float4 S = {st[0], st[Dv], st[2 * Dv], st[3 * Dv]};
  const int64_t step = static_cast<int64_t>(a.H) * D * Dv, qw = static_cast<int64_t>(a.H) * D;
  float* w = a.work + (static_cast<int64_t>(first) * a.H + h) * D * Dv + static_cast<int64_t>(e) * D + d;
  const float* b0 = a.sums + row0 * qw + h * D + d;
  for (int c0 = 0; c0 < chunks; c0 += kGlCarryFlight) {
    float4 u[kGlCarryFlight], b[kGlCarryFlight];
#pragma unroll
    for (int j = 0; j < kGlCarryFlight; ++j) {
      const int c = min(c0 + j, chunks - 1);
      u[j] = ld4<float>(w + c * step);
      b[j] = ld4<float>(b0 + (min((c + 1) * kChunkRows, rows) - 1) * qw);
    }
#pragma unroll
    for (int j = 0; j < kGlCarryFlight; ++j) {
      if (c0 + j < chunks) {
        st4<float>(w + (c0 + j) * step, S);
        S = float4{fmaf(__expf(b[j].x), S.x, u[j].x), fmaf(__expf(b[j].y), S.y, u[j].y), fmaf(__expf(b[j].z), S.z, u[j].z),
                   fmaf(__expf(b[j].w), S.w, u[j].w)};
      }
    }
  }
  st[0] = S.x; st[Dv] = S.y; st[2 * Dv] = S.z; st[3 * Dv] = S.w;
}

// The outputs of a chunk: wave w makes rows 16 w .. + 15 in all columns, norms them and applies the gate.
template <int NV>
__global__ __launch_bounds__(kGlThreads, NV <= 8 ? 2 : 1) void gated_linear_chunk_out_kernel(const GlChunkArgs a, const float* __restrict__ norm,
                                                                            float eps, void* __restrict__ out, int out_dtype) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const ChunkAt at = find_chunk(a.seg_row0, a.segments, blockIdx.x);
  if (at.rows == 0) return;
  const int h = blockIdx.y, tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, n = lane % 16, g = lane / 16;
  const int D = a.D, Dv = a.Dv;
  constexpr int EP = 16 * NV, vr = EP + 4;         // columns, those past Dv zero
  float* ks = lds;                                 // [64][68] k's slice, counted; behind the slices v [64][EP + 4] from here on
  float* ss = lds + kChunkRows * kGlSliceRow;      // [EP][68] the state's slice
  float* vs = lds;
  float* ps = lds + kChunkRows * vr;               // the masked P, [64][68]
  const int64_t qw = static_cast<int64_t>(a.H) * D;
  const float* y0 = a.y + at.row0 * a.row_stride + h * D;          // q's entries of the chunk's first row
  const float* b0 = a.sums + at.row0 * qw + h * D;
  const float* S0 = a.work + (static_cast<int64_t>(blockIdx.x) * a.H + h) * D * Dv;     // [e][d]
  const int blocks = (at.rows + 15) / 16;          // row blocks of sixteen that hold rows
  const int mine = min(16 * wave + n, at.rows - 1);                // this lane's row as an operand
  const float4 zero = {0.f, 0.f, 0.f, 0.f};
  f32x4_t p[4], o[NV];
#pragma unroll
  for (int j = 0; j < 4; ++j) p[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int j = 0; j < NV; ++j) o[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int d0 = 0; d0 < D; d0 += kGlSlice) {
    // fetched into registers first: the state's slice, k's slice with its sums, this lane's pieces of q and of its sums
    float4 s_next[NV], k_next[4], kb[4], ke[4], q4[4], b4[4];
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const int i = x * kGlThreads + tid, e = min(i / (kGlSlice / 4), Dv - 1), d = min(d0 + 4 * (i % (kGlSlice / 4)), D - 4);
      s_next[x] = ld4<float>(S0 + static_cast<int64_t>(e) * D + d);
    }
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int i = x * kGlThreads + tid, r = i / (kGlSlice / 4), d = min(d0 + 4 * (i % (kGlSlice / 4)), D - 4);
      const int rr = min(r, at.rows - 1), last = min(r / 16 * 16 + 15, at.rows - 1);
      k_next[x] = ld4<float>(y0 + rr * a.row_stride + qw + d);
      kb[x] = ld4<float>(b0 + rr * qw + d);
      ke[x] = ld4<float>(b0 + last * qw + d);
    }
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int d = min(d0 + 16 * x + 4 * g, D - 4);
      q4[x] = ld4<float>(y0 + mine * a.row_stride + d);
      b4[x] = ld4<float>(b0 + mine * qw + d);
    }
    __syncthreads();                               // the slice before has been read
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int i = x * kGlThreads + tid, r = i / (kGlSlice / 4), c = 4 * (i % (kGlSlice / 4));
      *reinterpret_cast<float4*>(&ks[r * kGlSliceRow + c]) =
          (r < at.rows && d0 + c < D) ? times_exp(k_next[x], ke[x], kb[x]) : zero;
    }
#pragma unroll
    for (int x = 0; x < NV; ++x) {                 // (past D the query's piece is zero, columns past Dv are dropped)
      const int i = x * kGlThreads + tid;
      *reinterpret_cast<float4*>(&ss[(i / (kGlSlice / 4)) * kGlSliceRow + 4 * (i % (kGlSlice / 4))]) = s_next[x];
    }
    __syncthreads();
    if (wave < blocks) {
      const bool row_in = 16 * wave + n < at.rows;
#pragma unroll
      for (int x = 0; x < 4; ++x)
        if (!(row_in && d0 + 16 * x + 4 * g < D)) q4[x] = zero;
      // the own block: may its queries' factor stay a factor?
      const float* own_end = b0 + min(16 * wave + 15, at.rows - 1) * qw;
      float grows = 0.f;
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const float4 e4 = ld4<float>(own_end + min(d0 + 16 * x + 4 * g, D - 4));
        grows = fmaxf(fmaxf(fmaxf(b4[x].x - e4.x, b4[x].y - e4.y), fmaxf(b4[x].z - e4.z, b4[x].w - e4.w)), grows);
      }
      const bool by_pairs = __any(grows > kGlMaxGrowth);
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const int c = 16 * x + 4 * g;
        const float4 qa = times_exp(q4[x], b4[x], zero);
#pragma unroll
        for (int j = 0; j < NV; ++j) o[j] = mfma4(qa, *reinterpret_cast<const float4*>(&ss[(16 * j + n) * kGlSliceRow + c]), o[j]);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          if (j < wave || (j == wave && !by_pairs)) {
            const float4 e4 = ld4<float>(b0 + min(16 * j + 15, at.rows - 1) * qw + min(d0 + c, D - 4));
            p[j] = mfma4(times_exp(q4[x], b4[x], e4), *reinterpret_cast<const float4*>(&ks[(16 * j + n) * kGlSliceRow + c]), p[j]);
          }
        }
      }
      if (by_pairs) {                              // rows 4 g + i of the block, key row n: one key entry after the other
        const int kj = min(16 * wave + n, at.rows - 1);
        float add[4] = {0.f, 0.f, 0.f, 0.f};
        for (int d = d0; d < min(d0 + kGlSlice, D); ++d) {
          const float kd = y0[kj * a.row_stride + qw + d], bj = b0[kj * qw + d];
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int qi = min(16 * wave + 4 * g + i, at.rows - 1);
            if (n <= 4 * g + i) add[i] = fmaf(y0[qi * a.row_stride + d] * kd, __expf(b0[qi * qw + d] - bj), add[i]);
          }
        }
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (j == wave) {
#pragma unroll
            for (int i = 0; i < 4; ++i) p[j][i] += add[i];
          }
      }
    }
  }
  float4 v_next[NV];                               // the chunk's values, 64 rows of EP entries over the workgroup
#pragma unroll
  for (int x = 0; x < NV; ++x) {
    const int i = x * kGlThreads + tid, r = min(i / (EP / 4), at.rows - 1), e = min(4 * (i % (EP / 4)), Dv - 4);
    v_next[x] = ld4<float>(a.y + (at.row0 + r) * a.row_stride + 2 * qw + h * Dv + e);
  }
  __syncthreads();                                 // the last slices have been read by every wave
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = 16 * wave + 4 * g + i;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = 16 * j + n;
      ps[r * kGlSliceRow + c] = c <= r ? p[j][i] : 0.f;
    }
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
    const int i = x * kGlThreads + tid, r = i / (EP / 4), e = 4 * (i % (EP / 4));
    *reinterpret_cast<float4*>(&vs[r * vr + e]) = (r < at.rows && e < Dv) ? v_next[x] : zero;
  }
  __syncthreads();
  if (wave >= blocks) return;
  for (int s = 0; s <= wave; ++s) {                // (a wave's own rows: what it wrote of ps it reads itself)
    const int r = 16 * s + 4 * g;
    const float4 pa = *reinterpret_cast<const float4*>(&ps[(16 * wave + n) * kGlSliceRow + r]);
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const float* vp = vs + r * vr + 16 * j + n;
      o[j] = mfma4(pa, float4{vp[0], vp[vr], vp[2 * vr], vp[3 * vr]}, o[j]);
    }
  }
  const float q_scale = 1.0f / sqrtf(static_cast<float>(D));
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = 16 * wave + 4 * g + i;
    float sq = 0.f;
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      o[j][i] *= q_scale;
      if (16 * j + n < Dv) sq = fmaf(o[j][i], o[j][i], sq);
    }
    const float inv = 1.0f / sqrtf(row_sum16(sq) / static_cast<float>(Dv) + eps);
    if (r >= at.rows) continue;
    const int64_t t = at.row0 + r;
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int e = 16 * j + n;
      if (e < Dv) store_from_float(out, out_dtype, (t * a.H + h) * Dv + e, o[j][i] * inv * norm[e] * gate_act(gates[i][j], kActSilu));
    }
  }
}

}  // namespace arle

using namespace arle;

// y float32: `parts` partial products part_stride apart of rows row_stride apart, columns q | k | v | gate | middle; one row a
// segment.  a2 [H * D, rank] of a2_dtype, a2_bias float32 [H * D], norm float32 [Dv].  out [T, H * Dv] of out_dtype.
extern "C" int arle_gated_linear_decode(const float* y, int parts, long long part_stride, long long row_stride, const void* a2,
                                        int a2_dtype, int rank, const float* a2_bias, float inv_tau, const float* norm,
                                        const int* seg_row0, const int* seg_slot, float* s_state, float eps, void* out,
                                        int out_dtype, int segments, int H, int D, int Dv, void* stream) {
  if (segments == 0) return 0;
  if (parts < 1 || H < 1 || H > 65535 || D < 1 || D > kGlMaxD || Dv < 4 || Dv > kGlMaxDv || Dv % 4 || rank < 1 || rank > kGlMaxRank ||
      reinterpret_cast<uintptr_t>(s_state) % 16)
    return static_cast<int>(hipErrorInvalidValue);
  hipStream_t s = static_cast<hipStream_t>(stream);
#define ARLE_GLD(TW)                                                                                                     \
  gated_linear_decode_kernel<TW><<<dim3(segments, H), kGlThreads, 0, s>>>(y, parts, part_stride, row_stride,             \
      static_cast<const TW*>(a2), rank, a2_bias, inv_tau, norm, seg_row0, seg_slot, s_state, eps, out, out_dtype, H, D, Dv)
  if (a2_dtype == kF32) ARLE_GLD(float); else ARLE_GLD(bf16);
#undef ARLE_GLD
  return launch_status();
}

// y float32 [T, .], columns q | k | v | gate.  sums float32 [T, H * D] (decay_gates).  work: float32 [items, H, Dv, D] with
// items at least the number of chunks of 64 rows of all segments.  out [T, H * Dv] of out_dtype.
extern "C" int arle_gated_linear_chunks(const float* y, long long row_stride, const float* sums, const int* seg_row0,
                                        const int* seg_slot, const float* norm, float* s_state, int segments, int items,
                                        float* work, float eps, void* out, int out_dtype, int H, int D, int Dv, void* stream) {
  if (segments == 0 || items == 0) return 0;
  auto al = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  if (H < 1 || H > 65535 || D < 4 || D > 256 || D % 4 || Dv < 4 || Dv > 256 || Dv % 4 || row_stride % 4 || !al(y) || !al(work) ||
      !al(sums))
    return static_cast<int>(hipErrorInvalidValue);
  const GlChunkArgs a{y, row_stride, sums, seg_row0, seg_slot, segments, s_state, work, H, D, Dv};
  hipStream_t s = static_cast<hipStream_t>(stream);
  const int DP = (D + 15) / 16 * 16;
  const int columns = Dv <= 64 ? 64 : (Dv <= 128 ? 128 : 256);
  const size_t sum_lds = static_cast<size_t>(kChunkRows) * (DP + 4 + columns + 4) * sizeof(float);
  const size_t slices = static_cast<size_t>(kChunkRows + columns) * kGlSliceRow, last = static_cast<size_t>(kChunkRows) * (columns + 4 + kGlSliceRow);
  const size_t out_lds = (slices > last ? slices : last) * sizeof(float);
  static bool raised = false;
  if (!raised) {
    const void* kernels[] = {reinterpret_cast<const void*>(&gated_linear_chunk_sum_kernel<4>),
                             reinterpret_cast<const void*>(&gated_linear_chunk_sum_kernel<8>),
                             reinterpret_cast<const void*>(&gated_linear_chunk_out_kernel<4>),
                             reinterpret_cast<const void*>(&gated_linear_chunk_out_kernel<8>),
                             reinterpret_cast<const void*>(&gated_linear_chunk_out_kernel<16>)};
    for (const void* f : kernels) {
      const hipError_t e = hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, 144 * 1024);
      if (e != hipSuccess) return static_cast<int>(e);
    }
    raised = true;
  }
  const dim3 grid(items, H);
  if (columns == 64)
    gated_linear_chunk_sum_kernel<4><<<grid, kGlThreads, sum_lds, s>>>(a);
  else
    gated_linear_chunk_sum_kernel<8><<<grid, kGlThreads, sum_lds, s>>>(a);
  gated_linear_chunk_carry_kernel<<<dim3(segments, H, (D / 4 * Dv + kGlThreads - 1) / kGlThreads), kGlThreads, 0, s>>>(a);
  if (columns == 64)
    gated_linear_chunk_out_kernel<4><<<grid, kGlThreads, out_lds, s>>>(a, norm, eps, out, out_dtype);
  else if (columns == 128)
    gated_linear_chunk_out_kernel<8><<<grid, kGlThreads, out_lds, s>>>(a, norm, eps, out, out_dtype);
  else
    gated_linear_chunk_out_kernel<16><<<grid, kGlThreads, out_lds, s>>>(a, norm, eps, out, out_dtype);
  return launch_status();
}
