// Attention of a latent layer on the matrix cores: all query heads share one key/value head whose keys are
// [c | k_rot] (D = C + R numbers a token) and whose values are c (see latent.hip), bfloat16 in, 32-bit scores, softmax
// and sums.
//
//   s_rj = scale * q_r . k_j  for the keys j <= pos(r), j > pos(r) - window;   p = softmax (a term exp(sink_h) in the
//   denominator, optional);   out_r = sum_j p_rj c_j          for every row r = (token, head)
//
// Rows of a step are the T * H pairs (token, head), a plain matrix [T * H, D], so a tile of rows is several heads of
// several tokens, and a tile of keys serves all of them.  Both kernels compute score tiles turned (keys down, rows
// across) with v_mfma_f32_32x32x16_bf16: a lane then owns one row, its share of the probabilities is the operand of the
// second product as it lies (row i of a key tile is the key with bits 2 and 3 of i exchanged), and the softmax needs
// one exchange with the lane 32 further.  The outputs accumulate turned too (C down, rows across).
//   * `portion`: a workgroup of four waves takes 128 rows; tiles of 64 keys and their turned values go through LDS once
//     for all of them.  Row blocks are dealt so that a compute unit's two workgroups are a long and a short one.
//   * `decode` (one row a request): a workgroup takes 32 heads of one request and every splits-th group of four tiles
//     of 32 keys, a tile a wave, both operands straight from the pages; waves add up through LDS, splits in `merge`.
// C a multiple of 32 up to 256, D - C a multiple of 16 up to 64, pages of a multiple of 16 keys.
#include "common.h"

namespace arle {

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef float f32x16_t __attribute__((ext_vector_type(16)));
typedef uint32_t u32x4_t __attribute__((ext_vector_type(4)));

constexpr int kLaThreads = 256;
constexpr int kLaRows = 128;     // rows of a workgroup of `portion`, 32 a wave
constexpr int kLaKeys = 64;      // keys of a tile of `portion`
constexpr float kLog2e = 1.4426950408889634f;

__device__ __forceinline__ int swap23(int i) { return (i & ~12) | ((i & 4) << 1) | ((i & 8) >> 1); }
__device__ __forceinline__ float other_half(float v) { return __shfl_xor(v, 32, kWave); }
__device__ __forceinline__ f32x16_t mfma32(u32x4_t a, u32x4_t b, f32x16_t c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, b), c, 0, 0, 0);
}
// the key of register i (0..15) of a score tile, within its 32
__device__ __forceinline__ int key_of(int i, int g) { return (i & 7) + 8 * g + 16 * (i >> 3); }

struct LatentArgs {
  const bf16* q;            // [T * H, D]
  bf16* out;                // [T * H, C]
  const bf16* k_pages;      // [pages, page, D]
  const bf16* v_pages;      // [pages, C, page]
  const int* table;         // [slots, table_stride]
  int table_stride;
  const int* seg_row0;
  const int* seg_slot;
  const int* seg_start;
  int segments;
  int H, D, C, page_shift;  // page size = 1 << page_shift
  float scale2;             // scale * log2(e)
  int window;               // 0: none
  const void* sink;         // [H] or null
  int sink_dtype;
};

// The values of eight keys from `key` on (a multiple of 8) for one c, those past `last` as zeros: a slot that holds no
// key yet may hold anything, and zero times that is not always zero.
__device__ __forceinline__ u32x4_t mask_values(u32x4_t v, int key, int last) {
  u32x4_t r;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    uint32_t w = v[i];
    if (key + 2 * i > last) w = 0;
    else if (key + 2 * i + 1 > last) w &= 0xffffu;
    r[i] = w;
  }
  return r;
}

// Sixteen bytes from memory to LDS at `dst` (the same in all lanes of the wave) + 16 * lane, past the registers.
__device__ __forceinline__ void load_to_lds(const bf16* src, bf16* dst) {
  __builtin_amdgcn_global_load_lds(src, (__attribute__((address_space(3))) void*)dst, 16, 0, 0);
}

// The same value, of which the compiler knows nothing: what is computed from it in a loop is computed there, not kept in
// registers across the loop.
__device__ __forceinline__ int unknown(int v) {
  asm volatile("" : "+v"(v));
  return v;
}

// A tile in LDS, in pieces of eight numbers: piece p of key row r lies at r * KP + (p ^ (r & 15)), piece p of value row c
// at c * 8 + (p ^ ((c >> 1) & 7)), so that the sixteen lanes that are served together never share a bank.
template <int NCT, int NDS>   // tiles of 32 of C; steps of 16 of D, of which those past D multiply zeros of the query
__global__ __launch_bounds__(kLaThreads, NCT <= 6 ? 2 : 1) void latent_attn_portion_kernel(const LatentArgs a) {
  constexpr int KP = (2 * NDS + 15) / 16 * 16;              // pieces a key row takes
  __shared__ __attribute__((aligned(16))) bf16 ks[kLaKeys * KP * 8];
  __shared__ __attribute__((aligned(16))) bf16 vs[NCT * 32 * kLaKeys];
  // which row block: of `total`, the first half of the workgroups takes them from the last (longest) on, the second half
  // from the first on
  int total = 0;
  for (int s = 0; s < a.segments; ++s) total += ((a.seg_row0[s + 1] - a.seg_row0[s]) * a.H + kLaRows - 1) / kLaRows;
  int item = blockIdx.x;
  if (item >= total) return;
  const int front = (total + 1) / 2;
  item = item < front ? total - 1 - item : item - front;
  int seg = 0;
  for (;; ++seg) {
    const int blocks = ((a.seg_row0[seg + 1] - a.seg_row0[seg]) * a.H + kLaRows - 1) / kLaRows;
    if (item < blocks) break;
    item -= blocks;
  }
  const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, n = lane % 32, g = lane / 32;
  const int rows = (a.seg_row0[seg + 1] - a.seg_row0[seg]) * a.H, start = a.seg_start[seg];
  const int r0 = item * kLaRows, last_row = min(r0 + kLaRows, rows) - 1;
  const int kmax = start + last_row / a.H;                                             // the last key anyone here sees
  const int kmin = a.window > 0 ? max(0, start + r0 / a.H - a.window + 1) : 0;         // and the first
  const int* table = a.table + static_cast<int64_t>(a.seg_slot[seg]) * a.table_stride;
  const int page = 1 << a.page_shift;
  const int r = min(r0 + 32 * wave + n, rows - 1);                                     // this lane's row (the last one again past the end)
  const int pos = start + r / a.H, low = a.window > 0 ? pos - a.window + 1 : 0;
  const int wave_max_pos = start + min(r0 + 32 * wave + 31, rows - 1) / a.H;
  const int wave_min_pos = start + min(r0 + 32 * wave, rows - 1) / a.H;
  const int64_t row = static_cast<int64_t>(a.seg_row0[seg]) * a.H + r;
  const int nds = a.D / 16, np = a.D / 8;
  u32x4_t qf[NDS];
#pragma unroll
  for (int s = 0; s < NDS; ++s) {
    const u32x4_t v = *reinterpret_cast<const u32x4_t*>(a.q + row * a.D + 16 * min(s, nds - 1) + 8 * g);
    qf[s] = s < nds ? v : u32x4_t{0, 0, 0, 0};
  }
  f32x16_t o[NCT];
#pragma unroll
  for (int c = 0; c < NCT; ++c)
#pragma unroll
    for (int i = 0; i < 16; ++i) o[c][i] = 0.f;
  float m = -INFINITY, l = 0.f;

  // the pages of a tile's four groups of sixteen keys, asked for a tile ahead; keys outside [kmin, kmax] are fetched as
  // the nearest one inside (their pages may be gone, or not there yet)
  auto inside = [&](int key) { return min(max(key, kmin), kmax); };
  int id0, id1, id2, id3;
  auto ask = [&](int t0) {
    id0 = table[inside(t0) >> a.page_shift];
    id1 = table[inside(t0 + 16) >> a.page_shift];
    id2 = table[inside(t0 + 32) >> a.page_shift];
    id3 = table[inside(t0 + 48) >> a.page_shift];
  };
  auto page_of = [&](int in_tile) {
    const int low_half = in_tile & 16 ? id1 : id0, high_half = in_tile & 16 ? id3 : id2;
    return in_tile & 32 ? high_half : low_half;
  };
  ask(kmin / kLaKeys * kLaKeys);
  for (int t0 = kmin / kLaKeys * kLaKeys; t0 <= kmax; t0 += kLaKeys) {
    const int id = unknown(tid), ln = id % 32, lg = id / 32 % 2;
    __syncthreads();                                        // the tile before has been read
    if (page >= kLaKeys && t0 >= kmin && t0 + kLaKeys - 1 <= kmax) {      // all of it in one page
      const int64_t first = static_cast<int64_t>(__builtin_amdgcn_readfirstlane(id0)) * page, off = t0 & (page - 1);
      const bf16* kbase = a.k_pages + (first + off) * a.D;
      const bf16* vbase = a.v_pages + first * a.C + off;
#pragma unroll
      for (int x = 0; x < kLaKeys * KP / kLaThreads; ++x) {
        const int at = x * kLaThreads + id, kr = at / KP, piece = min((at % KP) ^ (kr & 15), np - 1);
        load_to_lds(kbase + (kr * a.D + 8 * piece), ks + (x * kLaThreads + wave * kWave) * 8);
      }
#pragma unroll
      for (int x = 0; x < NCT; ++x) {
        const int at = x * kLaThreads + id, c = at / 8, piece = (at % 8) ^ ((c >> 1) & 7);
        load_to_lds(vbase + (c * page + 8 * piece), vs + (x * kLaThreads + wave * kWave) * 8);
      }
    } else {
#pragma unroll
      for (int x = 0; x < kLaKeys * KP / kLaThreads; ++x) {
        const int at = x * kLaThreads + id, kr = at / KP, piece = min((at % KP) ^ (kr & 15), np - 1);
        const int key = inside(t0 + kr);
        const int64_t slot = static_cast<int64_t>(page_of(key - t0)) * page + (key & (page - 1));
        load_to_lds(a.k_pages + slot * a.D + 8 * piece, ks + (x * kLaThreads + wave * kWave) * 8);
      }
#pragma unroll
      for (int x = 0; x < NCT; ++x) {
        const int at = x * kLaThreads + id, c = at / 8, piece = (at % 8) ^ ((c >> 1) & 7);
        const int key = min(max(t0 + 8 * piece, kmin & ~7), kmax & ~7);
        const int64_t line = static_cast<int64_t>(page_of(key - t0)) * a.C + c;
        load_to_lds(a.v_pages + line * page + (key & (page - 1)), vs + (x * kLaThreads + wave * kWave) * 8);
      }
    }
    if (t0 + kLaKeys <= kmax) ask(t0 + kLaKeys);
    __builtin_amdgcn_s_waitcnt(0);                          // every load that goes to LDS has arrived
    __syncthreads();
    if (t0 + kLaKeys - 1 > kmax) {                          // the last tile: slots behind the last key may hold anything
#pragma unroll
      for (int x = 0; x < NCT; ++x) {
        const int at = x * kLaThreads + tid, c = at / 8;
        const int key = min(max(t0 + 8 * ((at % 8) ^ ((c >> 1) & 7)), kmin & ~7), kmax & ~7);      // as it was fetched
        u32x4_t* v = reinterpret_cast<u32x4_t*>(&vs[at * 8]);
        if (key + 7 > kmax) *v = mask_values(*v, key, kmax);
      }
      __syncthreads();
    }
    if (t0 > wave_max_pos) continue;                        // (every wave keeps the barriers' count)
    const bool whole = t0 + kLaKeys - 1 <= wave_min_pos && (a.window == 0 || t0 > wave_max_pos - a.window);
    const int kr = swap23(ln);
#pragma unroll
    for (int h = 0; h < 2; ++h) {                           // 32 keys at a time
      f32x16_t s;
#pragma unroll
      for (int i = 0; i < 16; ++i) s[i] = 0.f;
      const bf16* krow = ks + (32 * h + kr) * KP * 8;
#pragma unroll
      for (int d = 0; d < NDS; ++d)
        s = mfma32(*reinterpret_cast<const u32x4_t*>(krow + ((2 * d + lg) ^ (kr & 15)) * 8), qf[d], s);
      float top = -INFINITY;
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        float v = s[i] * a.scale2;
        if (!whole) {
          const int key = t0 + 32 * h + key_of(i, g);
          if (key > pos || key < low) v = -INFINITY;
        }
        s[i] = v;
        top = fmaxf(top, v);
      }
      top = fmaxf(top, other_half(top));
      // the point that exponentials are taken from moves only when it has to: sums stay far below overflow
      if (__any(top > m + 8.f)) {
        const float m_new = fmaxf(m, top);
        const float f = m == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m - m_new);
        m = m_new;
        l *= f;
#pragma unroll
        for (int c = 0; c < NCT; ++c)
#pragma unroll
          for (int i = 0; i < 16; ++i) o[c][i] *= f;
      }
      const float from = m == -INFINITY ? 0.f : m;
      u32x4_t pf[2];
#pragma unroll
      for (int k = 0; k < 2; ++k)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float p0 = __builtin_amdgcn_exp2f(s[8 * k + 2 * i] - from), p1 = __builtin_amdgcn_exp2f(s[8 * k + 2 * i + 1] - from);
          l += p0 + p1;
          pf[k][i] = pack_bf16x2(p0, p1);
        }
      const bf16* vrow = vs + ln * kLaKeys;
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const int at = ((4 * h + 2 * k + lg) ^ ((ln >> 1) & 7)) * 8;
#pragma unroll
        for (int c = 0; c < NCT; ++c) o[c] = mfma32(*reinterpret_cast<const u32x4_t*>(vrow + 32 * c * kLaKeys + at), pf[k], o[c]);
      }
    }
  }
  l += other_half(l);
  if (a.sink) l += __builtin_amdgcn_exp2f(load_as_float(a.sink, a.sink_dtype, r % a.H) * kLog2e - m);
  if (r0 + 32 * wave + n >= rows) return;
  const float inv = 1.0f / l;
  bf16* orow = a.out + row * a.C + 4 * g;
#pragma unroll
  for (int c = 0; c < NCT; ++c)
#pragma unroll
    for (int i = 0; i < 16; i += 4)
      st4<bf16>(orow + 32 * c + 2 * i, float4{o[c][i] * inv, o[c][i + 1] * inv, o[c][i + 2] * inv, o[c][i + 3] * inv});
}

// parts: part_o float32 [segments, splits, H, C] unnormalised, part_ml [segments, splits, H, 2] (largest score, sum).
template <int NCT, int NDS>
__global__ __launch_bounds__(kLaThreads) void latent_attn_decode_kernel(const LatentArgs a, int splits, float* __restrict__ part_o,
                                                                        float* __restrict__ part_ml) {
  __shared__ __attribute__((aligned(16))) float os[2][NCT * 32 * 32];   // two waves' sums, [c / 4][row][4]
  __shared__ float ml[2][32][2];
  const int seg = blockIdx.x, split = blockIdx.y, h0 = blockIdx.z * 32;
  const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, n = lane % 32, g = lane / 32;
  const int pos = a.seg_start[seg], kmin = a.window > 0 ? max(0, pos - a.window + 1) : 0;
  const int* table = a.table + static_cast<int64_t>(a.seg_slot[seg]) * a.table_stride;
  const int page = 1 << a.page_shift, nds = a.D / 16;
  const int head = min(h0 + n, a.H - 1);
  const int64_t row = static_cast<int64_t>(a.seg_row0[seg]) * a.H + head;
  const int64_t part = (static_cast<int64_t>(seg) * splits + split) * a.H + h0 + n;
  const int first_tile = kmin / 32, tiles = pos / 32 - first_tile + 1;
  if (split * 4 >= tiles) {      // nothing for this workgroup: a part without weight
    if (tid < 32 && h0 + n < a.H) {
      part_ml[part * 2] = -INFINITY;
      part_ml[part * 2 + 1] = 0.f;
    }
    return;
  }
  u32x4_t qf[NDS];
#pragma unroll
  for (int s = 0; s < NDS; ++s) {
    const u32x4_t v = *reinterpret_cast<const u32x4_t*>(a.q + row * a.D + 16 * min(s, nds - 1) + 8 * g);
    qf[s] = s < nds ? v : u32x4_t{0, 0, 0, 0};
  }
  f32x16_t o[NCT];
#pragma unroll
  for (int c = 0; c < NCT; ++c)
#pragma unroll
    for (int i = 0; i < 16; ++i) o[c][i] = 0.f;
  float m = -INFINITY, l = 0.f;
  for (int tile = split * 4 + wave; tile < tiles; tile += 4 * splits) {
    const int t0 = (first_tile + tile) * 32;
    const int key = min(max(t0 + swap23(n), kmin), pos);
    const int64_t kpg = table[key >> a.page_shift];
    const bf16* krow = a.k_pages + (kpg * page + (key & (page - 1))) * a.D + 8 * g;
    const bf16* vrow[2];
    int vkey[2];
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      const int vk = vkey[k] = min(max(t0 + 16 * k + 8 * g, kmin & ~7), pos & ~7);
      const int64_t vpg = table[vk >> a.page_shift];
      vrow[k] = a.v_pages + (vpg * a.C + n) * page + (vk & (page - 1));
    }
    u32x4_t kf[NDS], vf[NCT][2];
#pragma unroll
    for (int s = 0; s < NDS; ++s) kf[s] = *reinterpret_cast<const u32x4_t*>(krow + 16 * min(s, nds - 1));
#pragma unroll
    for (int c = 0; c < NCT; ++c)
#pragma unroll
      for (int k = 0; k < 2; ++k) vf[c][k] = *reinterpret_cast<const u32x4_t*>(vrow[k] + static_cast<int64_t>(32 * c) * page);
    f32x16_t s;
#pragma unroll
    for (int i = 0; i < 16; ++i) s[i] = 0.f;
#pragma unroll
    for (int d = 0; d < NDS; ++d) s = mfma32(kf[d], qf[d], s);
    float top = -INFINITY;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int j = t0 + key_of(i, g);
      s[i] = (j > pos || j < kmin) ? -INFINITY : s[i] * a.scale2;
      top = fmaxf(top, s[i]);
    }
    top = fmaxf(top, other_half(top));
    const float m_new = fmaxf(m, top);      // (a tile holds at least one key that is seen)
    const float f = m == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m - m_new);
    m = m_new;
    l *= f;
    u32x4_t pf[2];
#pragma unroll
    for (int k = 0; k < 2; ++k)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float p0 = __builtin_amdgcn_exp2f(s[8 * k + 2 * i] - m), p1 = __builtin_amdgcn_exp2f(s[8 * k + 2 * i + 1] - m);
        l += p0 + p1;
        pf[k][i] = pack_bf16x2(p0, p1);
      }
    if (t0 + 31 > pos) {
#pragma unroll
      for (int c = 0; c < NCT; ++c)
#pragma unroll
        for (int k = 0; k < 2; ++k) vf[c][k] = mask_values(vf[c][k], vkey[k], pos);
    }
#pragma unroll
    for (int c = 0; c < NCT; ++c) {
#pragma unroll
      for (int i = 0; i < 16; ++i) o[c][i] *= f;
#pragma unroll
      for (int k = 0; k < 2; ++k) o[c] = mfma32(vf[c][k], pf[k], o[c]);
    }
  }
  l += other_half(l);
  // waves 2 and 3 into 0 and 1, then wave 1 into 0
#pragma unroll
  for (int step = 2; step > 0; step >>= 1) {
    if (wave >= step && wave < 2 * step) {
      const int w = wave - step;
      if (g == 0) {
        ml[w][n][0] = m;
        ml[w][n][1] = l;
      }
#pragma unroll
      for (int c = 0; c < NCT; ++c)
#pragma unroll
        for (int i = 0; i < 16; i += 4)
          *reinterpret_cast<float4*>(&os[w][((8 * c + i / 2 + g) * 32 + n) * 4]) = float4{o[c][i], o[c][i + 1], o[c][i + 2], o[c][i + 3]};
    }
    __syncthreads();
    if (wave < step) {
      const float m2 = ml[wave][n][0], l2 = ml[wave][n][1], m_new = fmaxf(m, m2);
      const float f1 = m == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m - m_new), f2 = m2 == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m2 - m_new);
      m = m_new;
      l = l * f1 + l2 * f2;
#pragma unroll
      for (int c = 0; c < NCT; ++c)
#pragma unroll
        for (int i = 0; i < 16; i += 4) {
          const float4 e = *reinterpret_cast<const float4*>(&os[wave][((8 * c + i / 2 + g) * 32 + n) * 4]);
          o[c][i] = fmaf(f2, e.x, f1 * o[c][i]); o[c][i + 1] = fmaf(f2, e.y, f1 * o[c][i + 1]);
          o[c][i + 2] = fmaf(f2, e.z, f1 * o[c][i + 2]); o[c][i + 3] = fmaf(f2, e.w, f1 * o[c][i + 3]);
        }
    }
    __syncthreads();
  }
  if (wave != 0 || h0 + n >= a.H) return;
  if (splits == 1) {
    if (a.sink) l += __builtin_amdgcn_exp2f(load_as_float(a.sink, a.sink_dtype, head) * kLog2e - m);
    const float inv = 1.0f / l;
    bf16* orow = a.out + row * a.C + 4 * g;
#pragma unroll
    for (int c = 0; c < NCT; ++c)
#pragma unroll
      for (int i = 0; i < 16; i += 4)
        st4<bf16>(orow + 32 * c + 2 * i, float4{o[c][i] * inv, o[c][i + 1] * inv, o[c][i + 2] * inv, o[c][i + 3] * inv});
    return;
  }
  if (g == 0) {
    part_ml[part * 2] = m;
    part_ml[part * 2 + 1] = l;
  }
  float* po = part_o + part * a.C + 4 * g;
#pragma unroll
  for (int c = 0; c < NCT; ++c)
#pragma unroll
    for (int i = 0; i < 16; i += 4) st4<float>(po + 32 * c + 2 * i, float4{o[c][i], o[c][i + 1], o[c][i + 2], o[c][i + 3]});
}

// One wave a (request, head): the splits' sums in order; a lane takes four of C (C <= 256).
__global__ __launch_bounds__(kWave) void latent_attn_merge_kernel(const LatentArgs a, int splits, const float* __restrict__ part_o,
                                                                  const float* __restrict__ part_ml) {
  const int seg = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const int64_t base = static_cast<int64_t>(seg) * splits * a.H + h;
  float m = -INFINITY, l = 0.f;
  if (lane < splits) {      // splits <= 64: a split a lane
    m = part_ml[(base + static_cast<int64_t>(lane) * a.H) * 2];
    l = part_ml[(base + static_cast<int64_t>(lane) * a.H) * 2 + 1];
  }
  const float top = wave_max(m);
  const float f = m == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m - top);
  float total = wave_sum(l * f);
  if (a.sink) total += __builtin_amdgcn_exp2f(load_as_float(a.sink, a.sink_dtype, h) * kLog2e - top);
  const int c = min(4 * lane, a.C - 4);
  float4 acc = {0.f, 0.f, 0.f, 0.f};
  const unsigned long long live = __ballot(f != 0.f);      // splits with weight; they are not all the first ones
  for (unsigned long long left = live; left;) {
    float4 e[4];
    float w[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const bool in = left != 0;
      const int s = in ? __builtin_ctzll(left) : 0;
      left &= left - (in ? 1 : 0);
      w[u] = in ? __shfl(f, s, kWave) : 0.f;
      e[u] = ld4<float>(part_o + (base + static_cast<int64_t>(in ? s : __builtin_ctzll(live)) * a.H) * a.C + c);
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      acc.x = fmaf(w[u], e[u].x, acc.x); acc.y = fmaf(w[u], e[u].y, acc.y);
      acc.z = fmaf(w[u], e[u].z, acc.z); acc.w = fmaf(w[u], e[u].w, acc.w);
    }
  }
  if (4 * lane >= a.C) return;
  const float inv = 1.0f / total;
  const int64_t row = static_cast<int64_t>(a.seg_row0[seg]) * a.H + h;
  st4<bf16>(a.out + row * a.C + c, float4{acc.x * inv, acc.y * inv, acc.z * inv, acc.w * inv});
}

}  // namespace arle

using namespace arle;

// q bf16 [T * H, D] and out bf16 [T * H, C], contiguous.  splits > 0: every segment is one row, `splits` (<= 64) parts of
// its keys with part_o, part_ml (see above; unused with one); splits == 0: row blocks of 128, `items` of them at most.
extern "C" int arle_latent_attn(const void* q, void* out, const void* k_pages, const void* v_pages, const int* table,
                                int table_stride, const int* seg_row0, const int* seg_slot, const int* seg_start, int segments,
                                int H, int D, int C, int page_size, float scale, int window, const void* sink, int sink_dtype,
                                int items, int splits, float* part_o, float* part_ml, void* stream) {
  if (segments == 0) return 0;
  const int R = D - C;
  if (H < 1 || H > 65535 || C < 32 || C > 256 || C % 32 || R < 0 || R > 64 || R % 16 || page_size < 16 ||
      (page_size & (page_size - 1)) || window < 0 || splits < 0 || splits > 64 || (splits > 1 && (!part_o || !part_ml)))
    return static_cast<int>(hipErrorInvalidValue);
  const LatentArgs a{static_cast<const bf16*>(q), static_cast<bf16*>(out), static_cast<const bf16*>(k_pages),
                     static_cast<const bf16*>(v_pages), table, table_stride, seg_row0, seg_slot, seg_start, segments, H, D, C,
                     __builtin_ctz(page_size), scale * kLog2e, window, sink, sink_dtype};
  hipStream_t s = static_cast<hipStream_t>(stream);
#define ARLE_LA_D(NCT, NDS)                                                                                            \
  do {                                                                                                                 \
    if (splits == 0)                                                                                                   \
      latent_attn_portion_kernel<NCT, NDS><<<items, kLaThreads, 0, s>>>(a);                                            \
    else                                                                                                               \
      latent_attn_decode_kernel<NCT, NDS><<<dim3(segments, splits, (H + 31) / 32), kLaThreads, 0, s>>>(a, splits, part_o, part_ml); \
  } while (0)
#define ARLE_LA(NCT)                                                                     \
  do {                                                                                   \
    if (R <= 32) ARLE_LA_D(NCT, 2 * NCT + 2); else ARLE_LA_D(NCT, 2 * NCT + 4);          \
  } while (0)
  switch (C / 32) {
    case 1: ARLE_LA(1); break;
    case 2: ARLE_LA(2); break;
    case 3: ARLE_LA(3); break;
    case 4: ARLE_LA(4); break;
    case 5: ARLE_LA(5); break;
    case 6: ARLE_LA(6); break;
    case 7: ARLE_LA(7); break;
    default: ARLE_LA(8); break;
  }
#undef ARLE_LA
#undef ARLE_LA_D
  if (splits > 1) latent_attn_merge_kernel<<<dim3(segments, H), kWave, 0, s>>>(a, splits, part_o, part_ml);
  return launch_status();
}
