// Preparation of the operands of an attention with rotary positions: per-head norms of q and k in front of or
// behind the rotation, the rotation itself in either pairing, and the write of keys and values into the pages.
//
// For every head of q and k of a row at position p (D entries, of which the first R rotate):
//   before:  x <- x / sqrt(mean(x^2) + eps) * w        (w given: one weight of D for all heads of q, one for k)
//   rotate:  the pair (u, v) = (x[i], x[i + R/2])  (halves)  or  (x[2i], x[2i + 1])  (interleaved), i < R/2,
//            becomes (u c - v s, v c + u s) with c = cos[p][i], s = sin[p][i] from float32 tables [positions, R/2]
//            (a scaling of the frequencies and a factor on both are part of the tables)
//   after:   x <- x / sqrt(mean(x^2) + eps)             (unit_after)
// q is changed in place, k goes to pages [page, nkv, slot, Dk], v as it is to pages [page, nkv, Dv, slot].
// `rotary_qkv_store_kernel`: one wave a (row, head); the head lies in LDS between the steps so that a lane finds its
// partner.  `rotary_qkv_store_x8_kernel` (bfloat16, head sizes that are multiples of 8, at most 512, and for the
// halves pairing R / 2 a multiple of 8): a lane takes eight consecutive entries by one 16-byte access, the 1 to 64
// lanes of a head add their squares by lane exchanges, a partner of the halves pairing is eight entries of another
// lane, one of the interleaved pairing lies in the lane itself; a wave is then several heads, and a row of a model
// of ordinary widths a dozen waves where the first kernel takes half a hundred, each a chain of dependent loads.
// All of it is 32-bit arithmetic on the values as the projection left them, the same for a row wherever it stands.
#include "common.h"

namespace arle {

constexpr int kRotMaxD = 1024;

template <typename T>
__global__ __launch_bounds__(kWave) void rotary_qkv_store_kernel(
    T* __restrict__ q, long long q_stride, const T* __restrict__ k, long long k_stride, const T* __restrict__ v,
    long long v_stride, const void* __restrict__ q_weight, const void* __restrict__ k_weight, int w_dtype, float eps,
    int unit_after, const float* __restrict__ cos_t, const float* __restrict__ sin_t, int R, int interleaved,
    const int* __restrict__ positions, const int* __restrict__ slot_of_token, const int* __restrict__ block_table,
    int table_stride, T* __restrict__ k_pages, T* __restrict__ v_pages, int nq, int nkv, int Dk, int Dv,
    int page_size) {
  __shared__ float head[kRotMaxD];
  const int64_t t = blockIdx.x;
  const int y = blockIdx.y, lane = threadIdx.x;
  const int pos = positions[t];
  if (y >= nq + nkv) {
    const int page = block_table[static_cast<int64_t>(slot_of_token[t]) * table_stride + pos / page_size];
    const int g = y - nq - nkv;
    T* dst = v_pages + (static_cast<int64_t>(page) * nkv + g) * Dv * page_size + pos % page_size;
    for (int d = lane; d < Dv; d += kWave) dst[static_cast<int64_t>(d) * page_size] = v[t * v_stride + g * Dv + d];
    return;
  }
  const bool is_q = y < nq;
  const int g = is_q ? y : y - nq;
  const T* src = is_q ? q + t * q_stride + g * Dk : k + t * k_stride + g * Dk;
  const void* weight = is_q ? q_weight : k_weight;
  float x[kRotMaxD / kWave];
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < kRotMaxD / kWave; ++j) {
    const int d = lane + j * kWave;
    if (j * kWave < Dk) {
      x[j] = to_float(src[min(d, Dk - 1)]);
      if (d < Dk) ss = fmaf(x[j], x[j], ss);
    }
  }
  if (weight) {
    const float f = 1.0f / sqrtf(wave_sum(ss) / static_cast<float>(Dk) + eps);
#pragma unroll
    for (int j = 0; j < kRotMaxD / kWave; ++j) {
      const int d = lane + j * kWave;
      if (j * kWave < Dk) x[j] = x[j] * f * load_as_float(weight, w_dtype, min(d, Dk - 1));
    }
  }
  if (R > 0) {
#pragma unroll
    for (int j = 0; j < kRotMaxD / kWave; ++j) {
      const int d = lane + j * kWave;
      if (j * kWave < Dk && d < Dk) head[d] = x[j];
    }
    __syncthreads();
    const int half = R / 2;
    const float* c_row = cos_t + static_cast<int64_t>(pos) * half;
    const float* s_row = sin_t + static_cast<int64_t>(pos) * half;
#pragma unroll
    for (int j = 0; j < kRotMaxD / kWave; ++j) {
      const int d = lane + j * kWave;
      if (j * kWave < R && d < R) {
        const bool first = interleaved ? (d % 2 == 0) : (d < half);
        const int i = interleaved ? d / 2 : (first ? d : d - half);
        const int partner = interleaved ? (d ^ 1) : (first ? d + half : d - half);
        const float c = c_row[i], s = s_row[i], other = head[partner];
        x[j] = first ? x[j] * c - other * s : x[j] * c + other * s;
      }
    }
  }
  float f = 1.0f;
  if (unit_after) {
    ss = 0.f;
#pragma unroll
    for (int j = 0; j < kRotMaxD / kWave; ++j) {
      const int d = lane + j * kWave;
      if (j * kWave < Dk && d < Dk) ss = fmaf(x[j], x[j], ss);
    }
    f = 1.0f / sqrtf(wave_sum(ss) / static_cast<float>(Dk) + eps);
  }
  T* dst;
  if (is_q) {
    dst = q + t * q_stride + g * Dk;
  } else {
    const int page = block_table[static_cast<int64_t>(slot_of_token[t]) * table_stride + pos / page_size];
    dst = k_pages + ((static_cast<int64_t>(page) * nkv + g) * page_size + pos % page_size) * Dk;
  }
#pragma unroll
  for (int j = 0; j < kRotMaxD / kWave; ++j) {
    const int d = lane + j * kWave;
    if (j * kWave < Dk && d < Dk) dst[d] = from_float<T>(x[j] * f);
  }
}

// What a step of decoded rows has in front of it: the 32-bit partial sums of the product that made q, k and v, a row's columns
// q | k | v, added in order and rounded on the way in.
struct QkvSums {
  const float* p;
  int parts;
  long long part_stride, row_stride;
};

// Eight consecutive entries of the sums' column `col`, rounded to bfloat16.
__device__ __forceinline__ uint4 summed8(const QkvSums& a, int64_t t, int col) {
  float s[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
  const float* p = a.p + t * a.row_stride + col;
  for (int i0 = 0; i0 < a.parts; i0 += 4) {
    float4 e[4][2];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const float* part = p + min(i0 + u, a.parts - 1) * a.part_stride;
      e[u][0] = ld4<float>(part);
      e[u][1] = ld4<float>(part + 4);
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const bool in = i0 + u < a.parts;
      s[0] += in ? e[u][0].x : 0.f; s[1] += in ? e[u][0].y : 0.f; s[2] += in ? e[u][0].z : 0.f; s[3] += in ? e[u][0].w : 0.f;
      s[4] += in ? e[u][1].x : 0.f; s[5] += in ? e[u][1].y : 0.f; s[6] += in ? e[u][1].z : 0.f; s[7] += in ? e[u][1].w : 0.f;
    }
  }
  return uint4{pack_bf16x2(s[0], s[1]), pack_bf16x2(s[2], s[3]), pack_bf16x2(s[4], s[5]), pack_bf16x2(s[6], s[7])};
}

// Values of a step of many rows: 64 rows of a kv head go through LDS, and each entry's 64 are written by one wave, side by
// side where the rows' positions follow one another (the pages hold an entry's tokens next to each other).
constexpr int kTurnRows = 64;

__global__ __launch_bounds__(256) void value_store_kernel(const bf16* __restrict__ v, long long v_stride,
                                                          const int* __restrict__ positions, const int* __restrict__ slot_of_token,
                                                          const int* __restrict__ block_table, int table_stride,
                                                          bf16* __restrict__ v_pages, int tokens, int nkv, int Dv, int page_size) {
  extern __shared__ uint16_t tile[];      // [64][Dv + 2]
  const int t0 = blockIdx.x * kTurnRows, g = blockIdx.y, units = Dv / 8, row = Dv + 2;
  const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
  for (int i = threadIdx.x; i < kTurnRows * units; i += 256) {
    const int r = i / units, u = i % units;
    const uint4 raw = *reinterpret_cast<const uint4*>(v + static_cast<int64_t>(min(t0 + r, tokens - 1)) * v_stride + g * Dv + 8 * u);
    uint32_t* dst = reinterpret_cast<uint32_t*>(tile + r * row + 8 * u);
    dst[0] = raw.x; dst[1] = raw.y; dst[2] = raw.z; dst[3] = raw.w;
  }
  const int t = min(t0 + lane, tokens - 1), pos = positions[t];
  const int page = block_table[static_cast<int64_t>(slot_of_token[t]) * table_stride + pos / page_size];
  uint16_t* out = reinterpret_cast<uint16_t*>(v_pages) + (static_cast<int64_t>(page) * nkv + g) * Dv * page_size + pos % page_size;
  __syncthreads();
  if (t0 + lane >= tokens) return;
  for (int d = wave; d < Dv; d += 4) out[static_cast<int64_t>(d) * page_size] = tile[lane * row + d];
}

// LPH: lanes of a head (a power of two, 8 LPH >= Dk).  A row's lanes: (nq + nkv) LPH for q and k, then Dv / 8 for
// every head of v.
template <int LPH, bool SUMS>
__global__ __launch_bounds__(256) void rotary_qkv_store_x8_kernel(
    bf16* __restrict__ q, long long q_stride, const bf16* __restrict__ k, long long k_stride, const bf16* __restrict__ v,
    long long v_stride, const void* __restrict__ q_weight, const void* __restrict__ k_weight, int w_dtype, float eps,
    int unit_after, const float* __restrict__ cos_t, const float* __restrict__ sin_t, int R, int interleaved,
    const int* __restrict__ positions, const int* __restrict__ slot_of_token, const int* __restrict__ block_table,
    int table_stride, bf16* __restrict__ k_pages, bf16* __restrict__ v_pages, int nq, int nkv, int Dk, int Dv,
    int page_size, const QkvSums sums) {
  const int64_t t = blockIdx.x;
  const int idx = blockIdx.y * 256 + threadIdx.x, lane = threadIdx.x % kWave;
  const int qk_lanes = (nq + nkv) * LPH, qk_padded = (qk_lanes + kWave - 1) / kWave * kWave, v_units = Dv / 8;
  const int pos = positions[t];
  const int page = block_table[static_cast<int64_t>(slot_of_token[t]) * table_stride + pos / page_size];
  if (idx >= qk_padded) {   // whole waves: the values' lanes begin with a wave
    const int e = idx - qk_padded;
    if (e >= nkv * v_units) return;
    const int g = e / v_units, u = e % v_units;
    uint4 raw;
    if constexpr (SUMS) raw = summed8(sums, t, (nq + nkv) * Dk + g * Dv + 8 * u);
    else raw = *reinterpret_cast<const uint4*>(v + t * v_stride + g * Dv + 8 * u);
    uint16_t* dst = reinterpret_cast<uint16_t*>(v_pages) +
                    ((static_cast<int64_t>(page) * nkv + g) * Dv + 8 * u) * page_size + pos % page_size;
    const uint32_t w[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
    for (int i = 0; i < 8; ++i) dst[static_cast<int64_t>(i) * page_size] = static_cast<uint16_t>(w[i / 2] >> (16 * (i % 2)));
    return;
  }
  // lanes behind the last head of k fill its wave: they exchange with the others and load and store nothing of their own
  const int y = min(idx / LPH, nq + nkv - 1), u = idx % LPH;
  const bool is_q = y < nq, live = idx < qk_lanes && 8 * u < Dk;
  const int g = is_q ? y : y - nq;
  const void* weight = is_q ? q_weight : k_weight;
  float x[8];
  {
    uint4 raw;
    if constexpr (SUMS) {
      raw = summed8(sums, t, y * Dk + (live ? 8 * u : 0));
    } else {
      const bf16* src = is_q ? q + t * q_stride + g * Dk : k + t * k_stride + g * Dk;
      raw = *reinterpret_cast<const uint4*>(src + (live ? 8 * u : 0));
    }
    const uint32_t w[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      x[2 * i] = live ? __uint_as_float(w[i] << 16) : 0.f;
      x[2 * i + 1] = live ? __uint_as_float(w[i] & 0xffff0000u) : 0.f;
    }
  }
  auto head_sum_sq = [&]() {
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) ss = fmaf(x[i], x[i], ss);
#pragma unroll
    for (int off = LPH / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off, kWave);
    return ss;
  };
  if (weight) {
    float wv[8];
    if (w_dtype == kF32) {
      const float4* w4 = reinterpret_cast<const float4*>(static_cast<const float*>(weight) + (live ? 8 * u : 0));
      const float4 lo = w4[0], hi = w4[1];
      wv[0] = lo.x; wv[1] = lo.y; wv[2] = lo.z; wv[3] = lo.w;
      wv[4] = hi.x; wv[5] = hi.y; wv[6] = hi.z; wv[7] = hi.w;
    } else {
      const uint4 raw = *reinterpret_cast<const uint4*>(static_cast<const bf16*>(weight) + (live ? 8 * u : 0));
      const uint32_t w[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        wv[2 * i] = __uint_as_float(w[i] << 16);
        wv[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
      }
    }
    const float f = 1.0f / sqrtf(head_sum_sq() / static_cast<float>(Dk) + eps);
#pragma unroll
    for (int i = 0; i < 8; ++i) x[i] = x[i] * f * wv[i];
  }
  if (R > 0) {
    const int half = R / 2;
    const float* c_row = cos_t + static_cast<int64_t>(pos) * half;
    const float* s_row = sin_t + static_cast<int64_t>(pos) * half;
    if (interleaved && half % 4 == 0) {      // four pairs a lane, whose angles are one access each
      const int e = min(4 * u, half - 4);
      const float4 c4 = ld4<float>(c_row + e), s4 = ld4<float>(s_row + e);
      const float c[4] = {c4.x, c4.y, c4.z, c4.w}, s[4] = {s4.x, s4.y, s4.z, s4.w};
      if (4 * u < half) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float a = x[2 * i], b = x[2 * i + 1];
          x[2 * i] = a * c[i] - b * s[i];
          x[2 * i + 1] = b * c[i] + a * s[i];
        }
      }
    } else if (interleaved) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int e = 4 * u + i;   // the pair's number
        if (e < half) {
          const float c = c_row[e], s = s_row[e], a = x[2 * i], b = x[2 * i + 1];
          x[2 * i] = a * c - b * s;
          x[2 * i + 1] = b * c + a * s;
        }
      }
    } else {
      const int hu = half / 8;   // lanes of a half
      const bool first = u < hu, turns = u < 2 * hu;
      const int partner = turns ? (first ? lane + hu : lane - hu) : lane;
      float other[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) other[i] = __shfl(x[i], partner, kWave);
      if (turns) {
        const int e0 = 8 * (first ? u : u - hu);
        float cs[8], sn[8];
#pragma unroll
        for (int k = 0; k < 2; ++k) {
          const float4 c4 = ld4<float>(c_row + e0 + 4 * k), s4 = ld4<float>(s_row + e0 + 4 * k);
          cs[4 * k] = c4.x; cs[4 * k + 1] = c4.y; cs[4 * k + 2] = c4.z; cs[4 * k + 3] = c4.w;
          sn[4 * k] = s4.x; sn[4 * k + 1] = s4.y; sn[4 * k + 2] = s4.z; sn[4 * k + 3] = s4.w;
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          const float c = cs[i], s = sn[i];
          x[i] = first ? x[i] * c - other[i] * s : x[i] * c + other[i] * s;
        }
      }
    }
  }
  float f = 1.0f;
  if (unit_after) f = 1.0f / sqrtf(head_sum_sq() / static_cast<float>(Dk) + eps);
  if (!live) return;
  bf16* dst = is_q ? q + t * q_stride + g * Dk + 8 * u
                   : k_pages + ((static_cast<int64_t>(page) * nkv + g) * page_size + pos % page_size) * Dk + 8 * u;
  uint4 raw;
  raw.x = pack_bf16x2(x[0] * f, x[1] * f);
  raw.y = pack_bf16x2(x[2] * f, x[3] * f);
  raw.z = pack_bf16x2(x[4] * f, x[5] * f);
  raw.w = pack_bf16x2(x[6] * f, x[7] * f);
  *reinterpret_cast<uint4*>(dst) = raw;
}

}  // namespace arle

using namespace arle;

extern "C" int arle_rotary_qkv_store(void* q, long long q_stride, const void* k, long long k_stride, const void* v,
                                     long long v_stride, int dtype, const void* q_weight, const void* k_weight,
                                     int w_dtype, float eps, int unit_after, const void* cos_t, const void* sin_t,
                                     int rotary_dim, int interleaved, const int* positions, const int* slot_of_token,
                                     const int* block_table, int table_stride, void* k_pages, void* v_pages, int tokens,
                                     int nq, int nkv, int Dk, int Dv, int page_size, void* stream) {
  if (tokens == 0) return 0;
  if (Dk > kRotMaxD || rotary_dim > Dk || rotary_dim % 2) return static_cast<int>(hipErrorInvalidValue);
  hipStream_t s = static_cast<hipStream_t>(stream);
  const auto aligned = [](const void* p, long long stride) { return reinterpret_cast<uintptr_t>(p) % 16 == 0 && stride % 8 == 0; };
  if (dtype != kF32 && Dk % 8 == 0 && Dk <= 512 && Dv % 8 == 0 && (interleaved || rotary_dim % 16 == 0) &&
      aligned(cos_t, 8) && aligned(sin_t, 8) && aligned(q_weight, 8) && aligned(k_weight, 8) && aligned(q, q_stride) && aligned(k, k_stride) && aligned(v, v_stride) && aligned(k_pages, 8)) {
    int lph = 1;
    while (8 * lph < Dk) lph *= 2;
    // a head's lanes lie in one wave (lph divides 64); the values' lanes start at the next multiple of 64
    const bool turned = tokens >= kTurnRows && Dv <= 512 && nkv <= 65535;     // the values in a launch of their own
    const int lanes = ((nq + nkv) * lph + 63) / 64 * 64 + (turned ? 0 : nkv * (Dv / 8));
    if ((lanes + 255) / 256 <= 65535) {
      if (turned) {
        const size_t lds = static_cast<size_t>(kTurnRows) * (Dv + 2) * sizeof(uint16_t);     // at most 64 KB
        static bool raised = false;
        if (!raised && lds > 48 * 1024) {
          const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&value_store_kernel),
                                                   hipFuncAttributeMaxDynamicSharedMemorySize, 80 * 1024);
          if (e != hipSuccess) return static_cast<int>(e);
          raised = true;
        }
        value_store_kernel<<<dim3((tokens + kTurnRows - 1) / kTurnRows, nkv), 256, lds, s>>>(
            static_cast<const bf16*>(v), v_stride, positions, slot_of_token, block_table, table_stride, static_cast<bf16*>(v_pages),
            tokens, nkv, Dv, page_size);
      }
      const dim3 grid(tokens, (lanes + 255) / 256);
#define ARLE_ROT_X8(LPH)                                                                                             \
  rotary_qkv_store_x8_kernel<LPH, false><<<grid, 256, 0, s>>>(                                                       \
      static_cast<bf16*>(q), q_stride, static_cast<const bf16*>(k), k_stride, static_cast<const bf16*>(v), v_stride, \
      q_weight, k_weight, w_dtype, eps, unit_after, static_cast<const float*>(cos_t),                                \
      static_cast<const float*>(sin_t), rotary_dim, interleaved, positions, slot_of_token, block_table,              \
      table_stride, static_cast<bf16*>(k_pages), static_cast<bf16*>(v_pages), nq, nkv, Dk, Dv, page_size, QkvSums{})
      switch (lph) {
        case 1: ARLE_ROT_X8(1); break;
        case 2: ARLE_ROT_X8(2); break;
        case 4: ARLE_ROT_X8(4); break;
        case 8: ARLE_ROT_X8(8); break;
        case 16: ARLE_ROT_X8(16); break;
        case 32: ARLE_ROT_X8(32); break;
        default: ARLE_ROT_X8(64); break;
      }
#undef ARLE_ROT_X8
      return launch_status();
    }
  }
  dim3 grid(tokens, nq + 2 * nkv);
  if (dtype == kF32) {
    rotary_qkv_store_kernel<float><<<grid, kWave, 0, s>>>(
        static_cast<float*>(q), q_stride, static_cast<const float*>(k), k_stride, static_cast<const float*>(v), v_stride,
        q_weight, k_weight, w_dtype, eps, unit_after, static_cast<const float*>(cos_t), static_cast<const float*>(sin_t),
        rotary_dim, interleaved, positions, slot_of_token, block_table, table_stride, static_cast<float*>(k_pages),
        static_cast<float*>(v_pages), nq, nkv, Dk, Dv, page_size);
  } else {
    rotary_qkv_store_kernel<bf16><<<grid, kWave, 0, s>>>(
        static_cast<bf16*>(q), q_stride, static_cast<const bf16*>(k), k_stride, static_cast<const bf16*>(v), v_stride,
        q_weight, k_weight, w_dtype, eps, unit_after, static_cast<const float*>(cos_t), static_cast<const float*>(sin_t),
        rotary_dim, interleaved, positions, slot_of_token, block_table, table_stride, static_cast<bf16*>(k_pages),
        static_cast<bf16*>(v_pages), nq, nkv, Dk, Dv, page_size);
  }
  return launch_status();
}

// The same from the 32-bit partial sums of the product (columns q | k | v from sums on), bfloat16: q goes to q_out [T, nq * Dk].
// Dk and Dv multiples of 8, Dk up to 512, pointers 16-byte aligned, strides multiples of 4; the halves pairing rotates a
// multiple of 16 entries.
extern "C" int arle_rotary_sums_store(const float* sums, int parts, long long part_stride, long long row_stride, void* q_out,
                                      const void* q_weight, const void* k_weight, int w_dtype, float eps, int unit_after,
                                      const void* cos_t, const void* sin_t, int rotary_dim, int interleaved,
                                      const int* positions, const int* slot_of_token, const int* block_table,
                                      int table_stride, void* k_pages, void* v_pages, int tokens, int nq, int nkv, int Dk,
                                      int Dv, int page_size, void* stream) {
  if (tokens == 0) return 0;
  const auto al = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  if (parts < 1 || Dk < 8 || Dk > 512 || Dk % 8 || Dv < 8 || Dv % 8 || rotary_dim < 0 || rotary_dim > Dk || rotary_dim % 2 ||
      (!interleaved && rotary_dim % 16) || part_stride % 4 || row_stride % 4 || !al(sums) || !al(q_out) || !al(k_pages) ||
      !al(cos_t) || !al(sin_t) || !al(q_weight) || !al(k_weight))
    return static_cast<int>(hipErrorInvalidValue);
  int lph = 1;
  while (8 * lph < Dk) lph *= 2;
  const int lanes = ((nq + nkv) * lph + 63) / 64 * 64 + nkv * (Dv / 8);
  if ((lanes + 255) / 256 > 65535) return static_cast<int>(hipErrorInvalidValue);
  const dim3 grid(tokens, (lanes + 255) / 256);
  hipStream_t s = static_cast<hipStream_t>(stream);
  const QkvSums a{sums, parts, part_stride, row_stride};
#define ARLE_ROT_SUMS(LPH)                                                                                            \
  rotary_qkv_store_x8_kernel<LPH, true><<<grid, 256, 0, s>>>(                                                         \
      static_cast<bf16*>(q_out), static_cast<long long>(nq) * Dk, nullptr, 0, nullptr, 0, q_weight, k_weight, w_dtype, eps, \
      unit_after, static_cast<const float*>(cos_t), static_cast<const float*>(sin_t), rotary_dim, interleaved, positions, \
      slot_of_token, block_table, table_stride, static_cast<bf16*>(k_pages), static_cast<bf16*>(v_pages), nq, nkv, Dk, Dv, \
      page_size, a)
  switch (lph) {
    case 1: ARLE_ROT_SUMS(1); break;
    case 2: ARLE_ROT_SUMS(2); break;
    case 4: ARLE_ROT_SUMS(4); break;
    case 8: ARLE_ROT_SUMS(8); break;
    case 16: ARLE_ROT_SUMS(16); break;
    case 32: ARLE_ROT_SUMS(32); break;
    default: ARLE_ROT_SUMS(64); break;
  }
#undef ARLE_ROT_SUMS
  return launch_status();
}
