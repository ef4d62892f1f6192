// A mixture of experts: the router, and the experts' products over the tokens that chose them.
//
//   z = W_r h + bias (32-bit sums; bias optional),  s = sigmoid(z), softmax(z) over all router outputs, or z itself;  the
//   `top` experts with the largest s + correction are chosen (ties: the lower index), where the experts form `groups`
//   equal groups of neighbours among the `keep` groups with the largest such number in them only (the others count as
//   minus infinity);  weight of a chosen expert = s / (sum of the chosen s + 1e-20) * scale, or without the division
//   s * scale; where s is z itself, the softmax over the chosen z * scale.
//   expert e: down_e (silu(gate_e h) * (up_e h)), or without a gate down_e (max(up_e h, 0)^2).  Router outputs past the
//   experts that have tensors stand for experts that hand back their input (`moe_identity` writes their rows).  The
//   router's kernel also makes the one number a token that a shared expert's output is multiplied by, sigmoid(w_s h),
//   where the caller has one.
//
// `moe_route`: one or four tokens a workgroup.  `moe_expert`: a workgroup takes one expert, 64 consecutive rows of the step
// and 64 output columns; it lists the rows of its 64 that chose the expert (in row order) and multiplies only those, so
// no step sorts anything and a launch's shape follows the number of rows alone.  The result of (token t, its k-th
// choice) lies at row t * top + k: the gate|up pass leaves the activation there, the down pass the expert's output,
// which the consumer weighs and adds in the order of k.  Every output is summed in one fixed order over K (chains
// of 16, added in ascending order), whatever else the step holds.  bfloat16 runs the matrix-core forms further down.
#include "common.h"

namespace arle {

constexpr int kMaxExpertsPerLane = 16;   // experts <= 64 * 16

struct Best {
  float v;
  int i;
};

// What the wave's lanes wrote to LDS before this, its lanes read behind it.
__device__ __forceinline__ void wave_lds_fence() { __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront"); }

__device__ __forceinline__ Best wave_best(Best b) {
#pragma unroll
  for (int off = kWave / 2; off > 0; off >>= 1) {
    const float ov = __shfl_xor(b.v, off, kWave);
    const int oi = __shfl_xor(b.i, off, kWave);
    if (ov > b.v || (ov == b.v && oi < b.i)) {
      b.v = ov;
      b.i = oi;
    }
  }
  return b;
}

struct RouteRule {
  int softmax;     // 0: s = sigmoid(z); 1: s = softmax(z); 2: s = z, and the weights are the softmax over the chosen z
  int groups;      // equal groups of neighbouring experts (1: no groups)
  int keep;        // groups among which the choice is made
  int normalize;   // 1: the chosen scores are divided by their sum
  float scale;
};

// A workgroup takes TOK tokens: their rows go to LDS as floats once; wave w computes the logits of experts w, w + waves,
// ... for all of them, a router row read once for the TOK (eight consecutive entries a lane and step where the width
// allows, one otherwise: an order that depends on the width alone); then wave k picks the `top` experts of token k one
// after the other.  EPL: experts a lane looks after (experts <= 64 * EPL).
template <typename T, typename TW, bool VEC, int THREADS, int TOK, int EPL>
__global__ __launch_bounds__(THREADS) void moe_route_kernel(const T* __restrict__ x, long long x_stride,
                                                            const TW* __restrict__ w, const void* __restrict__ bias,
                                                            int b_dtype, const void* __restrict__ correction, int c_dtype,
                                                            const TW* __restrict__ shared_w,
                                                            float* __restrict__ shared_gate, int* __restrict__ ids,
                                                            float* __restrict__ weights, int tokens, int width, int experts,
                                                            int top, const RouteRule rule) {
  // [TOK][width] the rows, then a token's [experts] scores, [experts] choice numbers and [groups]
  extern __shared__ float route_lds[];
  float* xs = route_lds;
  const int per_token = 2 * experts + rule.groups;
  float* numbers = route_lds + TOK * width;
  const int64_t t0 = static_cast<int64_t>(blockIdx.x) * TOK;
  const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
#pragma unroll
  for (int k = 0; k < TOK; ++k) {
    const T* row = x + min(t0 + k, static_cast<int64_t>(tokens) - 1) * x_stride;
    for (int i = threadIdx.x; i < width; i += THREADS) xs[k * width + i] = to_float(row[i]);
  }
  __syncthreads();
  for (int e = wave; e < experts + (shared_w ? 1 : 0); e += THREADS / kWave) {
    const TW* we = e < experts ? w + static_cast<int64_t>(e) * width : shared_w;
    float dot[TOK];
#pragma unroll
    for (int k = 0; k < TOK; ++k) dot[k] = 0.f;
    if (VEC) {
#pragma unroll 4
      for (int i = 8 * lane; i < width; i += 8 * kWave) {
        const float4 lo = ld4<TW>(we + i), hi = ld4<TW>(we + i + 4);
#pragma unroll
        for (int k = 0; k < TOK; ++k) {
          const float* xk = xs + k * width + i;
          const float4 a = *reinterpret_cast<const float4*>(xk), b = *reinterpret_cast<const float4*>(xk + 4);
          dot[k] = fmaf(a.x, lo.x, dot[k]); dot[k] = fmaf(a.y, lo.y, dot[k]); dot[k] = fmaf(a.z, lo.z, dot[k]); dot[k] = fmaf(a.w, lo.w, dot[k]);
          dot[k] = fmaf(b.x, hi.x, dot[k]); dot[k] = fmaf(b.y, hi.y, dot[k]); dot[k] = fmaf(b.z, hi.z, dot[k]); dot[k] = fmaf(b.w, hi.w, dot[k]);
        }
      }
    } else {
      for (int i = lane; i < width; i += kWave) {
        const float v = to_float(we[i]);
#pragma unroll
        for (int k = 0; k < TOK; ++k) dot[k] = fmaf(xs[k * width + i], v, dot[k]);
      }
    }
#pragma unroll
    for (int k = 0; k < TOK; ++k) {
      float z = wave_sum(dot[k]);
      if (lane != 0 || t0 + k >= tokens) continue;
      if (e == experts) {
        shared_gate[t0 + k] = 1.0f / (1.0f + expf(-z));
        continue;
      }
      if (bias) z += load_as_float(bias, b_dtype, e);
      numbers[k * per_token + e] = rule.softmax ? z : 1.0f / (1.0f + expf(-z));
    }
  }
  __syncthreads();
  // From here on wave k works for token k; what goes through LDS goes from a wave to itself.
  if (wave >= TOK || t0 + wave >= tokens) return;
  const int64_t t = t0 + wave;
  float* score = numbers + wave * per_token;
  float* pick = score + experts;
  float* group_best = pick + experts;
  float s[EPL], choice[EPL];
#pragma unroll
  for (int j = 0; j < EPL; ++j) {
    const int e = lane + j * kWave;
    s[j] = e < experts ? score[e] : (rule.softmax ? -INFINITY : 0.f);
  }
  if (rule.softmax == 1) {   // over all router outputs, in 32 bits: the largest logit taken off, one sum in a fixed order
    float top_z = -INFINITY;
#pragma unroll
    for (int j = 0; j < EPL; ++j) top_z = fmaxf(top_z, s[j]);
    top_z = wave_max(top_z);
    float sum = 0.f;
#pragma unroll
    for (int j = 0; j < EPL; ++j) {
      s[j] = lane + j * kWave < experts ? expf(s[j] - top_z) : 0.f;
      sum += s[j];
    }
    const float inv = 1.0f / wave_sum(sum);
#pragma unroll
    for (int j = 0; j < EPL; ++j) s[j] *= inv;
  }
#pragma unroll
  for (int j = 0; j < EPL; ++j) {
    const int e = lane + j * kWave;
    choice[j] = e < experts ? s[j] + (correction ? load_as_float(correction, c_dtype, e) : 0.f) : -INFINITY;
    if (e < experts) pick[e] = choice[j];
  }
  if (rule.groups > 1) {
    const int per = experts / rule.groups;
    wave_lds_fence();
    // a group's number is the largest choice number in it; lane l looks after the groups l, l + 64, ...
    float best[EPL];
#pragma unroll
    for (int j = 0; j < EPL; ++j) {
      const int g = lane + j * kWave;
      float b = -INFINITY;
      if (g < rule.groups)
        for (int i = 0; i < per; ++i) b = fmaxf(b, pick[g * per + i]);
      best[j] = b;
      if (g < rule.groups) group_best[g] = 0.f;   // 1 once the group is kept
    }
    wave_lds_fence();
    for (int k = 0; k < rule.keep; ++k) {
      Best b{-INFINITY, 0x7fffffff};
#pragma unroll
      for (int j = 0; j < EPL; ++j) {
        const int g = lane + j * kWave;
        if (g < rule.groups && best[j] != INFINITY && (best[j] > b.v || (best[j] == b.v && g < b.i))) {
          b.v = best[j];
          b.i = g;
        }
      }
      b = wave_best(b);
#pragma unroll
      for (int j = 0; j < EPL; ++j) {
        if (b.i == lane + j * kWave) {
          best[j] = INFINITY;   // taken
          group_best[b.i] = 1.f;
        }
      }
    }
    wave_lds_fence();
#pragma unroll
    for (int j = 0; j < EPL; ++j) {
      const int e = lane + j * kWave;
      if (e < experts && group_best[e / per] == 0.f) choice[j] = -INFINITY;
    }
  }
  float sum = 0.f, mine = 0.f;   // lane k keeps the k-th chosen score (top <= 64)
  int mine_id = 0;
  unsigned taken = 0;            // bit j: this lane's expert lane + 64 j has been chosen
  for (int k = 0; k < top; ++k) {
    Best b{-INFINITY, 0x7fffffff};
#pragma unroll
    for (int j = 0; j < EPL; ++j) {
      const int e = lane + j * kWave;
      if (e < experts && !(taken >> j & 1u) && (choice[j] > b.v || (choice[j] == b.v && e < b.i))) {
        b.v = choice[j];
        b.i = e;
      }
    }
    b = wave_best(b);
    float sv = 0.f;
#pragma unroll
    for (int j = 0; j < EPL; ++j) {
      if (b.i == lane + j * kWave) {
        sv = s[j];
        taken |= 1u << j;
      }
    }
    sv = __shfl(sv, b.i % kWave, kWave);
    sum += sv;
    if (lane == k) {
      mine = sv;
      mine_id = b.i;
    }
  }
  if (rule.softmax == 2) {   // the softmax over the chosen
    const float top_z = wave_max(lane < top ? mine : -INFINITY);
    const float e = lane < top ? expf(mine - top_z) : 0.f;
    const float total = wave_sum(e);
    if (lane < top) {
      ids[t * top + lane] = mine_id;
      weights[t * top + lane] = e / total * rule.scale;
    }
    return;
  }
  if (lane < top) {
    ids[t * top + lane] = mine_id;
    weights[t * top + lane] = (rule.normalize ? mine / (sum + 1e-20f) : mine) * rule.scale;
  }
}

// The rows of experts without tensors: where token t's k-th choice is a router output from `first` on, row t * top + k
// of out (float32 [T * top, width]) is the token's input itself.  One workgroup a token: it reads the row once and
// writes it for each such choice (most tokens have none, and their workgroups leave after reading `top` numbers).
template <typename T>
__global__ __launch_bounds__(256) void moe_identity_kernel(const T* __restrict__ x, long long x_stride,
                                                           const int* __restrict__ ids, float* __restrict__ out, int top,
                                                           int width, int first) {
  const int64_t t = blockIdx.x;
  unsigned long long which = 0;   // bit k: the k-th choice is such an expert (top <= 64)
  for (int k = 0; k < top; ++k) which |= static_cast<unsigned long long>(ids[t * top + k] >= first) << k;
  if (!which) return;
  const T* row = x + t * x_stride;
  for (int i = threadIdx.x; i < width; i += 256) {
    const float v = to_float(row[i]);
    for (unsigned long long left = which; left; left &= left - 1)
      out[(t * top + __builtin_ctzll(left)) * width + i] = v;
  }
}

constexpr int kEM = 64, kEN = 64, kEK = 16;
constexpr int kExpertThreads = 256;

// Which of an expert's products a launch makes.
//   kGateUp: w [experts, 2 N, K] (gate rows, then up rows), rows of x are tokens, out[(t top + k), n] = silu(g) u of type T
//   kUp:     w [experts, N, K], rows of x are tokens, out[(t top + k), n] = max(u, 0)^2 of type T
//   kDown:   w [experts, N, K], rows of x are t top + k, out float32 [(t top + k), n]
// in_scale (kGateUp, kUp): null, or a factor for every (token, choice) on the expert's input, which by linearity is one on
// the 32-bit sums in front of the activation.
constexpr int kDown = 0, kGateUp = 1, kUp = 2;

__device__ __forceinline__ float squared_relu(float u) {
  const float r = fmaxf(u, 0.f);
  return r * r;
}

template <typename T, int MODE>
__global__ __launch_bounds__(kExpertThreads) void moe_expert_kernel(const T* __restrict__ x, long long x_stride,
                                                                    const T* __restrict__ w, const int* __restrict__ ids,
                                                                    const float* __restrict__ in_scale, void* __restrict__ out,
                                                                    int tokens, int top, int N,
                                                                    int K) {
  constexpr bool GATE_UP = MODE == kGateUp, TOKENS = MODE != kDown;   // TOKENS: rows of x are tokens
  __shared__ int list_t[kEM], list_k[kEM];
  __shared__ int count;
  __shared__ float as[kEK][kEM + 4];
  __shared__ float ws[kEK][kEN + 4];
  __shared__ float us[GATE_UP ? kEK : 1][kEN + 4];
  const int e = blockIdx.z;
  const int n0 = blockIdx.y * kEN;
  if (threadIdx.x < kWave) {
    const int t = blockIdx.x * kEM + threadIdx.x;
    int slot = -1;
    if (t < tokens)
      for (int k = 0; k < top; ++k)
        if (ids[static_cast<int64_t>(t) * top + k] == e) slot = k;
    const unsigned long long chose = __ballot(slot >= 0);
    if (slot >= 0) {
      const int rank = __popcll(chose & ((1ull << threadIdx.x) - 1ull));
      list_t[rank] = t;
      list_k[rank] = slot;
    }
    if (threadIdx.x == 0) count = __popcll(chose);
  }
  __syncthreads();
  const int rows = count;
  if (rows == 0) return;
  const T* we = w + static_cast<int64_t>(e) * (GATE_UP ? 2 : 1) * N * K;
  const int tx = threadIdx.x % 16, ty = threadIdx.x / 16;
  float acc[4][4] = {}, acc_u[4][4] = {};
  for (int k0 = 0; k0 < K; k0 += kEK) {
#pragma unroll
    for (int i = 0; i < (kEM * kEK) / kExpertThreads; ++i) {
      const int idx = threadIdx.x + i * kExpertThreads;
      const int r = idx / kEK, c = idx % kEK;
      const int gk = k0 + c, gn = n0 + r;
      float av = 0.f;
      if (r < rows && gk < K) {
        const int64_t src = TOKENS ? list_t[r] : static_cast<int64_t>(list_t[r]) * top + list_k[r];
        av = to_float(x[src * x_stride + gk]);
      }
      as[c][r] = av;
      const bool in = gn < N && gk < K;
      ws[c][r] = in ? to_float(we[static_cast<int64_t>(gn) * K + gk]) : 0.f;
      if (GATE_UP) us[c][r] = in ? to_float(we[static_cast<int64_t>(N + gn) * K + gk]) : 0.f;
    }
    __syncthreads();
    float part[4][4] = {}, part_u[4][4] = {};
#pragma unroll
    for (int kk = 0; kk < kEK; ++kk) {
      float av[4], wv[4], uv[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) av[i] = as[kk][ty * 4 + i];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        wv[j] = ws[kk][tx * 4 + j];
        if (GATE_UP) uv[j] = us[kk][tx * 4 + j];
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          part[i][j] = fmaf(av[i], wv[j], part[i][j]);
          if (GATE_UP) part_u[i][j] = fmaf(av[i], uv[j], part_u[i][j]);
        }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        acc[i][j] += part[i][j];
        if (GATE_UP) acc_u[i][j] += part_u[i][j];
      }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = ty * 4 + i;
    if (r >= rows) continue;
    const int64_t item = static_cast<int64_t>(list_t[r]) * top + list_k[r], dst = item * N;
    const float f = MODE != kDown && in_scale ? in_scale[item] : 1.0f;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int n = n0 + tx * 4 + j;
      if (n >= N) continue;
      if (GATE_UP) {
        const float g = f * acc[i][j];
        static_cast<T*>(out)[dst + n] = from_float<T>(g / (1.0f + expf(-g)) * (f * acc_u[i][j]));
      } else if (MODE == kUp) {
        static_cast<T*>(out)[dst + n] = from_float<T>(squared_relu(f * acc[i][j]));
      } else {
        static_cast<float*>(out)[dst + n] = acc[i][j];
      }
    }
  }
}

// ---- matrix-core forms (bfloat16) ----------------------------------------------------------------
// `v_mfma_f32_16x16x32_bf16`: both operands are eight consecutive k a lane (row or column lane % 16, k from 8 (lane / 16)
// on), the result's lane holds rows 4 (lane / 16) .. + 3 of column lane % 16.  K a multiple of 8; rows 16-byte aligned.
typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef float f32x4_t __attribute__((ext_vector_type(4)));
typedef uint32_t u32x4_t __attribute__((ext_vector_type(4)));

// ---- few rows ------------------------------------------------------------------------------------
// With at most 64 tokens an expert has a few rows, and a launch lasts as long as its weights take to arrive.  A wave
// takes sixteen output columns and streams their weight rows (gate|up: the sixteen gate rows and the matching up rows)
// from memory straight into the A operand through a ring of registers; the rows that chose the expert lie in LDS, a slice
// of K at a time, as the B operand.
constexpr int kFewRing = 8;        // steps of 32 k in flight

template <int MODE, int MT>        // MT tiles of sixteen rows at most
__global__ __launch_bounds__(256) void moe_expert_few_kernel(const bf16* __restrict__ x, long long x_stride,
                                                             const bf16* __restrict__ w, const int* __restrict__ ids,
                                                             const float* __restrict__ in_scale, void* __restrict__ out,
                                                             int tokens, int top, int N, int K) {
  constexpr bool GATE_UP = MODE == kGateUp, TOKENS = MODE != kDown;
  constexpr int kSlice = 1024 / MT, kRow = kSlice + 8;       // K of a slice; what a row of it takes in LDS
  __shared__ int list_src[64], list_dst[64];
  __shared__ int count;
  __shared__ __attribute__((aligned(16))) bf16 xs[16 * MT * kRow];
  const int e = blockIdx.y, lane = threadIdx.x % kWave, wave = threadIdx.x / kWave, n = lane % 16, g = lane / 16;
  if (wave == 0) {
    int slot = -1;
    if (lane < tokens)
      for (int k = 0; k < top; ++k)
        if (ids[static_cast<int64_t>(lane) * top + k] == e) slot = k;
    const unsigned long long chose = __ballot(slot >= 0);
    if (slot >= 0) {
      const int rank = __popcll(chose & ((1ull << lane) - 1ull));
      list_src[rank] = TOKENS ? lane : lane * top + slot;
      list_dst[rank] = lane * top + slot;
    }
    if (lane == 0) count = __popcll(chose);
  }
  __syncthreads();
  const int rows = count;
  if (rows == 0) return;
  const int col0 = blockIdx.x * 64 + wave * 16;
  const bf16* we = w + static_cast<int64_t>(e) * (GATE_UP ? 2 : 1) * N * K;
  const bf16* wg = we + static_cast<int64_t>(min(col0 + n, N - 1)) * K;
  const bf16* wu = wg + (GATE_UP ? static_cast<int64_t>(N) * K : 0);
  const int steps = (K + 31) / 32, tiles = (rows + 15) / 16;
  u32x4_t ring[kFewRing], ring_u[GATE_UP ? kFewRing : 1];
  auto fetch = [&](int step, int at) {      // a piece past K is the last piece again; what multiplies it is zero
    const int k = min(32 * step + 8 * g, K - 8);
    ring[at] = *reinterpret_cast<const u32x4_t*>(wg + k);
    if (GATE_UP) ring_u[at] = *reinterpret_cast<const u32x4_t*>(wu + k);
  };
#pragma unroll
  for (int i = 0; i < kFewRing; ++i) fetch(i, i);
  f32x4_t acc[MT], acc_u[GATE_UP ? MT : 1];
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    acc[m] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    if (GATE_UP) acc_u[m] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  }
  const u32x4_t zero = {0, 0, 0, 0};
  for (int k0 = 0; k0 < K; k0 += kSlice) {
    __syncthreads();      // the slice before has been read
    for (int i = threadIdx.x; i < rows * (kSlice / 8); i += 256) {
      const int r = i / (kSlice / 8), c = 8 * (i % (kSlice / 8));
      *reinterpret_cast<u32x4_t*>(&xs[r * kRow + c]) =
          k0 + c < K ? *reinterpret_cast<const u32x4_t*>(x + static_cast<int64_t>(list_src[r]) * x_stride + k0 + c) : zero;
    }
    __syncthreads();
    const int last = min(steps, (k0 + kSlice) / 32);
    for (int s0 = k0 / 32; s0 < last; s0 += kFewRing) {
#pragma unroll
      for (int i = 0; i < kFewRing; ++i) {
        const bf16x8_t a = __builtin_bit_cast(bf16x8_t, ring[i]), u = __builtin_bit_cast(bf16x8_t, ring_u[GATE_UP ? i : 0]);
        fetch(s0 + i + kFewRing, i);
        const int c = 32 * (s0 + i) - k0 + 8 * g;
        if (s0 + i < last) {
#pragma unroll
          for (int m = 0; m < MT; ++m) {
            if (m < tiles) {
              const bf16x8_t b = __builtin_bit_cast(bf16x8_t, *reinterpret_cast<const u32x4_t*>(&xs[min(16 * m + n, rows - 1) * kRow + c]));
              acc[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, acc[m], 0, 0, 0);
              if (GATE_UP) acc_u[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(u, b, acc_u[m], 0, 0, 0);
            }
          }
        }
      }
    }
  }
  // acc[m][i]: output column 4 g + i of the wave's sixteen, listed row 16 m + n
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const int r = 16 * m + n;
    if (r >= rows) continue;
    const int64_t dst = static_cast<int64_t>(list_dst[r]) * N;
    const float f = MODE != kDown && in_scale ? in_scale[list_dst[r]] : 1.0f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int col = col0 + 4 * g + i;
      if (col >= N) continue;
      const float z = f * acc[m][i];
      if (GATE_UP)
        static_cast<bf16*>(out)[dst + col] = from_float<bf16>(z / (1.0f + expf(-z)) * (f * acc_u[GATE_UP ? m : 0][i]));
      else if (MODE == kUp)
        static_cast<bf16*>(out)[dst + col] = from_float<bf16>(squared_relu(z));
      else
        static_cast<float*>(out)[dst + col] = z;
    }
  }
}

// ---- many rows ------------------------------------------------------------------------------------
// With a few hundred rows an expert what a launch waits for is the passes over the weights: every workgroup streams its
// weight tile over all of K.  Here a workgroup of RG x 4 waves (RG 1 or 2) looks through RG x 256 rows of the step and takes RG x 64 listed rows and 256 weight rows
// (128 gate and the 128 matching up columns, or 256 columns of down) a k step, both through LDS: the weight tile is
// fetched once for all RG groups of 64 rows, and a wave multiplies the 64 rows of its group by 64 weight rows (32
// gate and their 32 up columns): sixteen products for four row and four weight fragments, twice a k step of 64.  Two
// k steps of loads are in flight; sixteen rows that hold no listed row are not multiplied.  (A k step of 64 instead
// of 32, with half the barriers a product: 4,647 instead of 5,228 us for the sixteen launches of a 2,048-token prefill
// at the Qwen3-4B widths.)
constexpr int kBigCols = 256;       // weight rows of a tile
constexpr int kBigRows = 64;        // listed rows of a group of four waves

template <int MODE, int RG, int BK>
__global__ __launch_bounds__(256 * RG) void moe_expert_tiles_kernel(const bf16* __restrict__ x, long long x_stride,
                                                                    const bf16* __restrict__ w, const int* __restrict__ ids,
                                                                    const float* __restrict__ in_scale, void* __restrict__ out,
                                                                    int tokens, int top, int N,
                                                                    int K) {
  constexpr bool GATE_UP = MODE == kGateUp, TOKENS = MODE != kDown;   // TOKENS: rows of x are tokens
  constexpr int kThreads = 256 * RG, kWaves = 4 * RG, kRows = kBigRows * RG;
  constexpr int kLdsRow = BK + 8;                 // bfloat16 a row of BK takes in LDS (no two lanes of a read on one bank)
  constexpr int kLanesRow = BK / 8;               // lanes that copy one row of a tile, a piece of 8 each (whole lines)
  constexpr int kPass = kThreads / kLanesRow;     // rows that the workgroup copies in one go
  constexpr int kWPieces = kBigCols / kPass, kAPieces = kRows / kPass;
  __shared__ int list_src[kThreads], list_dst[kThreads];
  __shared__ int wave_count[kWaves];
  __shared__ __attribute__((aligned(16))) bf16 wt[kBigCols * kLdsRow];
  __shared__ __attribute__((aligned(16))) bf16 at[kRows * kLdsRow];
  const int e = blockIdx.z;
  const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave, n = lane % 16, g = lane / 16;
  const int rg = wave / 4, cw = wave % 4;     // the wave's group of 64 rows, and its 64 weight rows of the tile
  {
    const int t = blockIdx.x * kThreads + threadIdx.x;
    int slot = -1;
    if (t < tokens)
      for (int k = 0; k < top; ++k)
        if (ids[static_cast<int64_t>(t) * top + k] == e) slot = k;
    const unsigned long long chose = __ballot(slot >= 0);
    if (lane == 0) wave_count[wave] = __popcll(chose);
    __syncthreads();
    int before = 0;
    for (int i = 0; i < wave; ++i) before += wave_count[i];
    if (slot >= 0) {
      const int rank = before + __popcll(chose & ((1ull << lane) - 1ull));
      list_src[rank] = TOKENS ? t : t * top + slot;
      list_dst[rank] = t * top + slot;
    }
    __syncthreads();
  }
  int rows = 0;
#pragma unroll
  for (int i = 0; i < kWaves; ++i) rows += wave_count[i];
  if (rows == 0) return;
  const int cols = GATE_UP ? kBigCols / 2 : kBigCols;     // output columns of the tile
  const int n0 = blockIdx.y * cols;
  const bf16* we = w + static_cast<int64_t>(e) * (GATE_UP ? 2 : 1) * N * K;
  // the weight rows of which this thread copies one piece of 8 into LDS: LDS row r belongs to column wave r / 64; of
  // its 64 rows the first 32 are gate columns, the last 32 the matching up columns
  const int piece = (static_cast<int>(threadIdx.x) % kLanesRow) * 8, prow = static_cast<int>(threadIdx.x) / kLanesRow;
  const bf16* wsrc[kWPieces];
  bool w_in[kWPieces];
#pragma unroll
  for (int h = 0; h < kWPieces; ++h) {
    const int r = kPass * h + prow;
    int wcol, wrow_global;
    if (GATE_UP) {
      const int within = r % 64;
      wcol = n0 + (r / 64) * 32 + within % 32;
      wrow_global = within < 32 ? wcol : N + wcol;
    } else {
      wcol = n0 + r;
      wrow_global = wcol;
    }
    w_in[h] = wcol < N;
    wsrc[h] = we + static_cast<int64_t>(w_in[h] ? wrow_global : 0) * K + piece;
  }
  const u32x4_t zero = {0, 0, 0, 0};
  for (int sub = 0; sub * kRows < rows; ++sub) {
    const bf16* asrc[kAPieces];
#pragma unroll
    for (int h = 0; h < kAPieces; ++h)
      asrc[h] = x + static_cast<int64_t>(list_src[min(sub * kRows + kPass * h + prow, rows - 1)]) * x_stride + piece;
    f32x4_t acc[4][4];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[i][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const int first = sub * kRows + kBigRows * rg;        // the first listed row of this wave's group
    const int live = max(0, min(4, (rows - first + 15) / 16));
    // two k steps are in flight: the loads of step k + 2 are sent while step k is multiplied
    u32x4_t a_set[2][kAPieces], w_set[2][kWPieces];
    auto fetch = [&](int k0, u32x4_t (&a_to)[kAPieces], u32x4_t (&w_to)[kWPieces]) {
#pragma unroll
      for (int h = 0; h < kAPieces; ++h)
        a_to[h] = k0 + piece < K ? *reinterpret_cast<const u32x4_t*>(asrc[h] + k0) : zero;
#pragma unroll
      for (int h = 0; h < kWPieces; ++h)
        w_to[h] = (w_in[h] && k0 + piece < K) ? *reinterpret_cast<const u32x4_t*>(wsrc[h] + k0) : zero;
    };
    auto step = [&](int k0, u32x4_t (&a_reg)[kAPieces], u32x4_t (&w_reg)[kWPieces]) {
      __syncthreads();      // the tiles before have been read by every wave
#pragma unroll
      for (int h = 0; h < kAPieces; ++h) *reinterpret_cast<u32x4_t*>(&at[(kPass * h + prow) * kLdsRow + piece]) = a_reg[h];
#pragma unroll
      for (int h = 0; h < kWPieces; ++h) *reinterpret_cast<u32x4_t*>(&wt[(kPass * h + prow) * kLdsRow + piece]) = w_reg[h];
      __syncthreads();
      if (k0 + 2 * BK < K) fetch(k0 + 2 * BK, a_reg, w_reg);
      if (live == 0) return;
#pragma unroll
      for (int kk = 0; kk < BK; kk += 32) {
        bf16x8_t a_op[4], b_op[4];
#pragma unroll
        for (int i = 0; i < 4; ++i)
          a_op[i] = __builtin_bit_cast(bf16x8_t, *reinterpret_cast<const u32x4_t*>(&at[(kBigRows * rg + 16 * i + n) * kLdsRow + kk + 8 * g]));
#pragma unroll
        for (int j = 0; j < 4; ++j)
          b_op[j] = __builtin_bit_cast(bf16x8_t, *reinterpret_cast<const u32x4_t*>(&wt[(64 * cw + 16 * j + n) * kLdsRow + kk + 8 * g]));
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (i < live) {       // sixteen rows of the 64 that hold no listed row are not multiplied
#pragma unroll
            for (int j = 0; j < 4; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a_op[i], b_op[j], acc[i][j], 0, 0, 0);
          }
      }
    };
    fetch(0, a_set[0], w_set[0]);
    if (BK < K) fetch(BK, a_set[1], w_set[1]);
    for (int k0 = 0; k0 < K; k0 += 2 * BK) {
      step(k0, a_set[0], w_set[0]);
      if (k0 + BK < K) step(k0 + BK, a_set[1], w_set[1]);
    }
    // acc[i][j][c]: listed row 16 i + 4 g + c of the group's 64, weight row 16 j + n of the wave's 64
#pragma unroll
    for (int i = 0; i < 4; ++i) {
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        const int rr = first + 16 * i + 4 * g + c;
        if (rr >= rows) continue;
        const int64_t dst = static_cast<int64_t>(list_dst[rr]) * N;
        const float f = MODE != kDown && in_scale ? in_scale[list_dst[rr]] : 1.0f;
        if (GATE_UP) {
#pragma unroll
          for (int j = 0; j < 2; ++j) {
            const int col = n0 + cw * 32 + 16 * j + n;
            const float gt = f * acc[i][j][c];
            if (col < N) static_cast<bf16*>(out)[dst + col] = from_float<bf16>(gt / (1.0f + expf(-gt)) * (f * acc[i][j + 2][c]));
          }
        } else {
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const int col = n0 + cw * 64 + 16 * j + n;
            if (col >= N) continue;
            if (MODE == kUp)
              static_cast<bf16*>(out)[dst + col] = from_float<bf16>(squared_relu(f * acc[i][j][c]));
            else
              static_cast<float*>(out)[dst + col] = acc[i][j][c];
          }
        }
      }
    }
    __syncthreads();        // before the next rows overwrite the tiles
  }
}

}  // namespace arle

using namespace arle;

// x [T, width] of x_dtype, w [experts, width] of w_dtype, bias and correction [experts] or null; shared_w [width] of
// w_dtype with shared_gate float32 [T], or null; ids int32 [T, top], weights float32 [T, top].
extern "C" int arle_moe_route(const void* x, long long x_stride, int x_dtype, const void* w, int w_dtype,
                              const void* bias, int b_dtype, const void* correction, int c_dtype, const void* shared_w,
                              float* shared_gate, int* ids, float* weights, int tokens, int width, int experts, int top,
                              float scale, int softmax, int groups, int keep, int normalize,
                              void* stream) {
  if (tokens == 0) return 0;
  if (softmax < 0 || softmax > 2 || (shared_w && !shared_gate)) return static_cast<int>(hipErrorInvalidValue);
  if (experts < 1 || experts > kWave * kMaxExpertsPerLane || top < 1 || top > experts || top > kWave || groups < 1 ||
      experts % groups || keep < 1 || keep > groups || top > keep * (experts / groups))
    return static_cast<int>(hipErrorInvalidValue);
  hipStream_t s = static_cast<hipStream_t>(stream);
  const RouteRule rule{softmax, groups, keep, normalize, scale};
  const bool vec = width % 8 == 0 && reinterpret_cast<uintptr_t>(w) % 16 == 0 && reinterpret_cast<uintptr_t>(shared_w) % 16 == 0;
  // many tokens share each router row four at a time; few are latency, a wave an expert
  const auto bytes = [&](int tok) { return static_cast<size_t>(tok) * (width + 2 * experts + groups) * sizeof(float); };
  const int tok = tokens > 128 && bytes(4) <= 80 * 1024 ? 4 : 1;
  const size_t lds = bytes(tok);
  if (lds > 80 * 1024) return static_cast<int>(hipErrorInvalidValue);
#define ARLE_ROUTE_K(TX, TWT, V, TH, TK, EPL)                                                                          \
  do {                                                                                                                 \
    static bool raised = false;                                                                                        \
    if (!raised && lds > 48 * 1024) {                                                                                  \
      const hipError_t err = hipFuncSetAttribute(reinterpret_cast<const void*>(&moe_route_kernel<TX, TWT, V, TH, TK, EPL>), \
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, 80 * 1024);               \
      if (err != hipSuccess) return static_cast<int>(err);                                                             \
      raised = true;                                                                                                   \
    }                                                                                                                  \
    moe_route_kernel<TX, TWT, V, TH, TK, EPL><<<(tokens + TK - 1) / TK, TH, lds, s>>>(                                 \
        static_cast<const TX*>(x), x_stride, static_cast<const TWT*>(w), bias, b_dtype, correction, c_dtype,           \
        static_cast<const TWT*>(shared_w), shared_gate, ids, weights, tokens, width, experts, top, rule);              \
  } while (0)
#define ARLE_ROUTE_T(TX, TWT, V, EPL)                          \
  do {                                                         \
    if (tok == 4) ARLE_ROUTE_K(TX, TWT, V, 256, 4, EPL);       \
    else ARLE_ROUTE_K(TX, TWT, V, 1024, 1, EPL);               \
  } while (0)
#define ARLE_ROUTE_V(TX, TWT, V)                                        \
  do {                                                                  \
    if (experts <= kWave) ARLE_ROUTE_T(TX, TWT, V, 1);                  \
    else if (experts <= 4 * kWave) ARLE_ROUTE_T(TX, TWT, V, 4);         \
    else ARLE_ROUTE_T(TX, TWT, V, kMaxExpertsPerLane);                  \
  } while (0)
#define ARLE_ROUTE(TX, TWT)                          \
  do {                                               \
    if (vec) ARLE_ROUTE_V(TX, TWT, true);            \
    else ARLE_ROUTE_V(TX, TWT, false);               \
  } while (0)
  if (x_dtype == kF32) {
    if (w_dtype == kF32) ARLE_ROUTE(float, float); else ARLE_ROUTE(float, bf16);
  } else {
    if (w_dtype == kF32) ARLE_ROUTE(bf16, float); else ARLE_ROUTE(bf16, bf16);
  }
#undef ARLE_ROUTE
#undef ARLE_ROUTE_V
#undef ARLE_ROUTE_T
#undef ARLE_ROUTE_K
  return launch_status();
}

// x [T, width] of `dtype`, ids int32 [T * top], out float32 [T * top, width]: see moe_identity_kernel.
extern "C" int arle_moe_identity(const void* x, long long x_stride, int dtype, const int* ids, void* out, int tokens,
                                 int top, int width, int first, void* stream) {
  if (tokens == 0) return 0;
  if (top < 1 || top > 64 || width < 1 || first < 0) return static_cast<int>(hipErrorInvalidValue);
  hipStream_t s = static_cast<hipStream_t>(stream);
  const unsigned items = static_cast<unsigned>(tokens);
  if (dtype == kF32)
    moe_identity_kernel<float><<<items, 256, 0, s>>>(static_cast<const float*>(x), x_stride, ids, static_cast<float*>(out), top, width, first);
  else
    moe_identity_kernel<bf16><<<items, 256, 0, s>>>(static_cast<const bf16*>(x), x_stride, ids, static_cast<float*>(out), top, width, first);
  return launch_status();
}

// mode: kGateUp, kUp or kDown (see above); in_scale float32 [T, top] or null; out [T * top, N] of `dtype`, or of float32 for kDown.
extern "C" int arle_moe_expert(const void* x, long long x_stride, const void* w, const int* ids, const float* in_scale,
                               void* out, int dtype,
                               int mode, int tokens, int experts, int top, int N, int K, void* stream) {
  if (tokens == 0) return 0;
  if (mode < 0 || mode > 2 || experts < 1 || experts > 65535 || top < 1 || N < 1 || K < 1 || (N + kEN - 1) / kEN > 65535)
    return static_cast<int>(hipErrorInvalidValue);
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (dtype == kBF16 && K % 8 == 0 && x_stride % 8 == 0 && reinterpret_cast<uintptr_t>(x) % 16 == 0 &&
      reinterpret_cast<uintptr_t>(w) % 16 == 0) {
    if (tokens > 64) {      // rows enough that an expert's list fills tiles of 64
      const int bcols = mode == kGateUp ? kBigCols / 2 : kBigCols;
      const bf16* xb = static_cast<const bf16*>(x);
      const bf16* wb = static_cast<const bf16*>(w);
#define ARLE_TILES(GU, RGS)                                                                                      \
  moe_expert_tiles_kernel<GU, RGS, 64><<<dim3((tokens + 256 * RGS - 1) / (256 * RGS), (N + bcols - 1) / bcols, experts), \
                                         256 * RGS, 0, s>>>(xb, x_stride, wb, ids, in_scale, out, tokens, top, N, K)
#define ARLE_TILES_MODE(RGS)              \
  do {                                    \
    if (mode == kGateUp)                  \
      ARLE_TILES(kGateUp, RGS);           \
    else if (mode == kUp)                 \
      ARLE_TILES(kUp, RGS);               \
    else                                  \
      ARLE_TILES(kDown, RGS);             \
  } while (0)
      // two groups of 64 rows a weight tile once the step has rows for them: a tile's fetch is what the launch waits
      // for (all sixteen launches of a 2,048-token prefill at the Qwen3-4B widths: one group 6,508 us, two 5,219 us,
      // four, which leaves a wave 128 registers, 5,456 us)
      if (tokens > 256) {
        ARLE_TILES_MODE(2);
      } else {
        ARLE_TILES_MODE(1);
      }
#undef ARLE_TILES_MODE
#undef ARLE_TILES
      return launch_status();
    }
    const dim3 fgrid((N + 63) / 64, experts);
#define ARLE_FEW(MODE, MT)                                                                                            \
  moe_expert_few_kernel<MODE, MT><<<fgrid, 256, 0, s>>>(static_cast<const bf16*>(x), x_stride, static_cast<const bf16*>(w), \
                                                        ids, in_scale, out, tokens, top, N, K)
#define ARLE_FEW_MT(MODE)          \
  do {                             \
    if (tokens <= 16)              \
      ARLE_FEW(MODE, 1);           \
    else if (tokens <= 32)         \
      ARLE_FEW(MODE, 2);           \
    else                           \
      ARLE_FEW(MODE, 4);           \
  } while (0)
    if (mode == kGateUp) ARLE_FEW_MT(kGateUp); else if (mode == kUp) ARLE_FEW_MT(kUp); else ARLE_FEW_MT(kDown);
#undef ARLE_FEW_MT
#undef ARLE_FEW
    return launch_status();
  }
  const dim3 grid((tokens + kEM - 1) / kEM, (N + kEN - 1) / kEN, experts);
#define ARLE_EXPERT(TT, GU)                                                                                         \
  moe_expert_kernel<TT, GU><<<grid, kExpertThreads, 0, s>>>(static_cast<const TT*>(x), x_stride,                    \
                                                            static_cast<const TT*>(w), ids, in_scale, out, tokens, top, N, K)
#define ARLE_EXPERT_MODE(TT)              \
  do {                                    \
    if (mode == kGateUp)                  \
      ARLE_EXPERT(TT, kGateUp);           \
    else if (mode == kUp)                 \
      ARLE_EXPERT(TT, kUp);               \
    else                                  \
      ARLE_EXPERT(TT, kDown);             \
  } while (0)
  if (dtype == kF32) ARLE_EXPERT_MODE(float); else ARLE_EXPERT_MODE(bf16);
#undef ARLE_EXPERT_MODE
#undef ARLE_EXPERT
  return launch_status();
}
