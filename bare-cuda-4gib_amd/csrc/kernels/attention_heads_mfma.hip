// Softmax attention on the matrix cores that keeps 32-bit queries, scores and weights: queries are float32, the cache is
// bfloat16 (keys [page, kv_head, token, dim], values [page, kv_head, token, vdim], as attention_maps.hip reads it), and every
// float operand -- a query's elements, a key's weight -- is handed to the matrix cores as three bfloat16 numbers whose sum it is
// exactly (the float's leading, middle and trailing eight bits).  A product of two bfloat16 numbers is exact in float32, so
// scores and weighted sums are float32 sums of exact products: what plain float arithmetic computes, in another order.
//
// For many rows of one request (a prompt portion).  A wave is 16 rows (tokens x query heads that share a key/value head),
// a workgroup four waves with consecutive rows that walk their keys together, 64 a tile (32 for large heads):
//   staging   the tile's keys and values pass from memory through registers, asked for a tile ahead, into LDS as they lie
//   scores    S^T = K Q^T: a lane holds, for its row, four keys of every 16
//   softmax   running maximum and sum of a row: in-lane and two lane swaps
//   output    O^T += V^T P^T: the scores' registers are the operand's as they lie; V^T comes through LDS's transposing read
// A row at position p sees key j <= p with p - j < window (window 0: every key); a sink exp(sink[head]) may join the
// denominator; the head's output is multiplied by a factor.  Keys outside the rows' common range are never read (their
// pages may be gone).  The workgroups of one key/value head follow each other eight apart, so that with eight of them an XCD's
// cache holds one head's keys; the longest walks start first.
#include <math.h>

#include "api.h"
#include "mfma.h"

namespace bc4g {
namespace {

constexpr int kRowsAWave = 16, kWavesAGroup = 4, kRowsAGroup = kRowsAWave * kWavesAGroup, kThreads = kWavesAGroup * kWave;
constexpr float kLog2E = 1.4426950408889634f;

typedef short shortx4 __attribute__((ext_vector_type(4)));

struct HeadsArgs {
  const float* q;
  long q_row;
  const bf16_t *k_cache, *v_cache;
  const int32_t* block_table;
  int table_stride;
  const int32_t *seq_start, *seq_ctx;
  void* out;
  int out_dtype;
  long out_row;
  int n_heads, n_kv_heads, dim, vdim, page_tokens, page_shift, window, n_tiles, wide_out;
  float scale, factor;
  const float* sink;
};

// Eight floats as three bfloat16 operands whose sum they are: each part takes the upper half of what the parts before left.
__device__ inline void split_three(const float (&x)[8], uint4 (&part)[3]) {
  float left[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) left[e] = x[e];
#pragma unroll
  for (int p = 0; p < 3; ++p) {
    uint32_t w[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const uint32_t lo = __float_as_uint(left[2 * e]), hi = __float_as_uint(left[2 * e + 1]);
      w[e] = __builtin_amdgcn_perm(hi, lo, 0x07060302u);
      if (p < 2) {
        left[2 * e] -= __uint_as_float(lo & 0xffff0000u);
        left[2 * e + 1] -= __uint_as_float(hi & 0xffff0000u);
      }
    }
    part[p] = make_uint4(w[0], w[1], w[2], w[3]);
  }
}

// maximum / sum of a value over the four lanes l, l ^ 16, l ^ 32, l ^ 48, in every lane
__device__ inline float four_lanes_max(float x) {
  const unsigned u = __float_as_uint(x);
  const auto a = __builtin_amdgcn_permlane16_swap(u, u, false, false);
  const float y = fmaxf(__uint_as_float(a[0]), __uint_as_float(a[1]));
  const unsigned v = __float_as_uint(y);
  const auto b = __builtin_amdgcn_permlane32_swap(v, v, false, false);
  return fmaxf(__uint_as_float(b[0]), __uint_as_float(b[1]));
}
__device__ inline float four_lanes_sum(float x) {
  const unsigned u = __float_as_uint(x);
  const auto a = __builtin_amdgcn_permlane16_swap(u, u, false, false);
  const float y = __uint_as_float(a[0]) + __uint_as_float(a[1]);
  const unsigned v = __float_as_uint(y);
  const auto b = __builtin_amdgcn_permlane32_swap(v, v, false, false);
  return __uint_as_float(b[0]) + __uint_as_float(b[1]);
}

// DS: 32-wide steps of the keys' dimensions (dim <= 32 DS), EB: blocks of 16 values (vdim <= 16 EB), KT: keys of a tile.
template <int DS, int EB, int KT>
__global__ __launch_bounds__(kThreads, (DS <= 4 && EB <= 4) || (DS <= 2 && EB <= 8) ? 3 : 2) void attention_heads_mfma_kernel(const HeadsArgs a) {
  constexpr int KB = KT / 16, KW = DS * 32 + 8, VW = EB * 16 + 16;        // (rows padded: the reads of 16 rows side by side meet different banks)
  constexpr int KP = DS * 4, VP = EB * 2;                                  // 16-byte pieces of a key's row, of a value's
  constexpr int KN = (KT * KP + kThreads - 1) / kThreads, VN = (KT * VP + kThreads - 1) / kThreads;
  __shared__ __align__(16) bf16_t k_s[KT][KW];
  __shared__ __align__(16) bf16_t v_s[KT][VW];
  const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, c = lane % 16, g = lane / 16;
  const int kvh = blockIdx.x % a.n_kv_heads, tile = a.n_tiles - 1 - blockIdx.x / a.n_kv_heads, s = blockIdx.y;
  const int hg = a.n_heads / a.n_kv_heads, start = a.seq_start[s], ctx = a.seq_ctx[s];
  const int rows = (a.seq_start[s + 1] - start) * hg, r0 = tile * kRowsAGroup;
  if (r0 >= rows) return;
  const int32_t* table = a.block_table + static_cast<long>(s) * a.table_stride;
  const int group_last = ctx + (min(r0 + kRowsAGroup, rows) - 1) / hg;                     // the positions of the group's rows
  const int group_first = ctx + r0 / hg;
  const int lo = a.window > 0 && group_first - a.window + 1 > 0 ? group_first - a.window + 1 : 0;

  // this lane's row (a lane beyond the last row repeats it and is dropped at the end), and the range of the wave's positions
  const int row = min(r0 + wave * kRowsAWave + c, rows - 1);
  const bool live = r0 + wave * kRowsAWave + c < rows;
  const int head = kvh * hg + row % hg, pos = ctx + row / hg;
  const long token = start + row / hg;
  const int wave_first = ctx + min(r0 + wave * kRowsAWave, rows - 1) / hg, wave_last = ctx + min(r0 + wave * kRowsAWave + 15, rows - 1) / hg;
  const int wave_lo = a.window > 0 ? wave_first - a.window + 1 : 0;

  uint4 qf[DS][3];
#pragma unroll
  for (int st = 0; st < DS; ++st) {
    const int d0 = st * 32 + 8 * g;
    float x[8] = {};
    if (d0 < a.dim) {
      const float* from = a.q + token * a.q_row + static_cast<long>(head) * a.dim + d0;
      const float4 x0 = *reinterpret_cast<const float4*>(from), x1 = *reinterpret_cast<const float4*>(from + 4);
      x[0] = x0.x, x[1] = x0.y, x[2] = x0.z, x[3] = x0.w, x[4] = x1.x, x[5] = x1.y, x[6] = x1.z, x[7] = x1.w;
    }
    split_three(x, qf[st]);
  }
  floatx4 o[EB];
#pragma unroll
  for (int eb = 0; eb < EB; ++eb) o[eb] = floatx4{0.f, 0.f, 0.f, 0.f};
  float m = -1e30f, l = 0.f;                                 // (m in powers of two; l: this lane's share of the row's sum)
  const float by = a.scale * kLog2E;

  uint4 k_next[KN], v_next[VN];
  auto row_of = [&](int j) -> long {                         // where key j lies among all tokens of the pool, for this key/value head
    const int page = a.page_shift >= 0 ? j >> a.page_shift : j / a.page_tokens;
    return (static_cast<long>(table[page]) * a.n_kv_heads + kvh) * a.page_tokens + (j - page * a.page_tokens);
  };
  auto fetch = [&](int j0) {
#pragma unroll
    for (int i = 0; i < KN; ++i) {
      const int idx = tid + i * kThreads, j = j0 + idx / KP, d = idx % KP * 8;
      k_next[i] = idx < KT * KP && j >= lo && j <= group_last && d < a.dim ? load16(a.k_cache + row_of(j) * a.dim + d) : zero16();
    }
#pragma unroll
    for (int i = 0; i < VN; ++i) {
      const int idx = tid + i * kThreads, j = j0 + idx / VP, d = idx % VP * 8;
      v_next[i] = idx < KT * VP && j >= lo && j <= group_last && d < a.vdim ? load16(a.v_cache + row_of(j) * a.vdim + d) : zero16();
    }
  };
  fetch(lo - lo % KT);
  for (int j0 = lo - lo % KT; j0 <= group_last; j0 += KT) {
    __syncthreads();                                         // (the tile before has been read)
#pragma unroll
    for (int i = 0; i < KN; ++i) {
      const int idx = tid + i * kThreads;
      if (idx < KT * KP) *reinterpret_cast<uint4*>(&k_s[idx / KP][idx % KP * 8]) = k_next[i];
    }
#pragma unroll
    for (int i = 0; i < VN; ++i) {
      const int idx = tid + i * kThreads;
      if (idx < KT * VP) *reinterpret_cast<uint4*>(&v_s[idx / VP][idx % VP * 8]) = v_next[i];
    }
    __syncthreads();
    if (j0 + KT <= group_last) fetch(j0 + KT);
    if (j0 > wave_last || j0 + KT <= wave_lo) continue;      // (no row of this wave sees a key of the tile)

    floatx4 sc[KB];
#pragma unroll
    for (int kb = 0; kb < KB; ++kb) {
      sc[kb] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int st = 0; st < DS; ++st) {
        const uint4 kf = load16(&k_s[16 * kb + c][32 * st + 8 * g]);
#pragma unroll
        for (int p = 2; p >= 0; --p) sc[kb] = mfma_16x16x32(kf, qf[st][p], sc[kb]);
      }
    }
    // (a tile that every row of the wave sees whole needs no mask)
    const bool whole = j0 + KT - 1 <= wave_first && (a.window <= 0 || j0 > wave_last - a.window);
    float top = m;
#pragma unroll
    for (int kb = 0; kb < KB; ++kb)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        float x = sc[kb][i] * by;
        if (!whole) {
          const int j = j0 + 16 * kb + 4 * g + i;
          if (j > pos || (a.window > 0 && pos - j >= a.window)) x = -INFINITY;
        }
        sc[kb][i] = x;
        top = fmaxf(top, x);
      }
    top = four_lanes_max(top);
    const float alpha = __builtin_amdgcn_exp2f(m - top);
    m = top;
    float sum = 0.f;
    uint4 pf[KT / 32][3];
#pragma unroll
    for (int h = 0; h < KT / 32; ++h) {
      float p[8];                                            // keys 4 g .. 4 g + 3 of the half's first 16, then of its second
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        p[i] = __builtin_amdgcn_exp2f(sc[2 * h + i / 4][i % 4] - top);
        sum += p[i];
      }
      split_three(p, pf[h]);
    }
    l = l * alpha + sum;
    if (__any(alpha != 1.0f)) {
#pragma unroll
      for (int eb = 0; eb < EB; ++eb) o[eb] *= alpha;
    }
#pragma unroll
    for (int h = 0; h < KT / 32; ++h)
#pragma unroll
      for (int eb = 0; eb < EB; ++eb) {
        // the transposing read: a group of 16 lanes points at four rows of 16 values and gets, lane by lane, a column of four
        const bf16_t* from = &v_s[32 * h + 4 * g + c / 4][16 * eb + 4 * (c % 4)];
        const shortx4 v0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) shortx4*)from);
        const shortx4 v1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) shortx4*)(from + 16 * VW));
        const uint2 u0 = __builtin_bit_cast(uint2, v0), u1 = __builtin_bit_cast(uint2, v1);
        const uint4 vf = make_uint4(u0.x, u0.y, u1.x, u1.y);
#pragma unroll
        for (int p = 2; p >= 0; --p) o[eb] = mfma_16x16x32(vf, pf[h][p], o[eb]);
      }
  }
  l = four_lanes_sum(l);
  float shrink = 1.0f;
  if (a.sink) {                                              // a term of the denominator, with no value
    const float sk = a.sink[head] * kLog2E, top = fmaxf(m, sk);
    shrink = __builtin_amdgcn_exp2f(m - top);
    l = l * shrink + __builtin_amdgcn_exp2f(sk - top);
  }
  if (!live) return;
  const float mult = shrink * a.factor / l;
#pragma unroll
  for (int eb = 0; eb < EB; ++eb) {
    const int e0 = 16 * eb + 4 * g;
    if (e0 >= a.vdim) continue;
    const long at = token * a.out_row + static_cast<long>(head) * a.vdim + e0;
    if (a.out_dtype == kF32) {
#pragma unroll
      for (int i = 0; i < 4; ++i) static_cast<float*>(a.out)[at + i] = o[eb][i] * mult;
    } else {
      uint32_t b[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) b[i] = bf16_bits_from_float(o[eb][i] * mult);
      bf16_t* to = static_cast<bf16_t*>(a.out) + at;
      if (a.wide_out) {
        *reinterpret_cast<uint2*>(to) = make_uint2(b[0] | (b[1] << 16), b[2] | (b[3] << 16));
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i) to[i].bits = static_cast<uint16_t>(b[i]);
      }
    }
  }
}

template <int DS, int EB>
void launch_heads(const HeadsArgs& a, dim3 grid, hipStream_t s) {
  constexpr int KT = DS <= 4 && EB <= 8 ? 64 : 32;
  attention_heads_mfma_kernel<DS, EB, KT><<<grid, kThreads, 0, s>>>(a);
}

template <int DS>
void launch_heads_values(const HeadsArgs& a, dim3 grid, hipStream_t s) {
  if (a.vdim <= 32) launch_heads<DS, 2>(a, grid, s);
  else if (a.vdim <= 64) launch_heads<DS, 4>(a, grid, s);
  else if (a.vdim <= 128) launch_heads<DS, 8>(a, grid, s);
  else launch_heads<DS, 16>(a, grid, s);
}

}  // namespace
}  // namespace bc4g

using namespace bc4g;

extern "C" int bc4g_attention_heads_mfma(const float* q, long q_row, const void* k_cache, const void* v_cache, const int32_t* block_table,
                                         int table_stride, const int32_t* seq_start, const int32_t* seq_ctx, int n_seqs, int most_rows,
                                         void* out, int out_dtype, long out_row, int n_heads, int n_kv_heads, int dim, int vdim,
                                         int page_tokens, int window, float scale, const float* sink, float factor, void* stream) {
  BC4G_REQUIRE(n_seqs >= 0 && n_seqs <= 65535 && most_rows >= 0 && n_heads > 0 && n_kv_heads > 0 && n_heads % n_kv_heads == 0,
               "attention_heads_mfma: bad sizes S=%d rows=%d heads=%d/%d", n_seqs, most_rows, n_heads, n_kv_heads);
  BC4G_REQUIRE(dim > 0 && dim <= 256 && dim % 8 == 0 && vdim > 0 && vdim <= 256 && vdim % 8 == 0,
               "attention_heads_mfma: dim=%d and vdim=%d must be multiples of 8 up to 256", dim, vdim);
  BC4G_REQUIRE(page_tokens > 0 && table_stride > 0 && window >= 0, "attention_heads_mfma: bad cache sizes page_tokens=%d table_stride=%d window=%d",
               page_tokens, table_stride, window);
  BC4G_REQUIRE(q && k_cache && v_cache && block_table && seq_start && seq_ctx && out && (out_dtype == kF32 || out_dtype == kBF16) &&
               q_row >= static_cast<long>(n_heads) * dim && q_row % 4 == 0 && out_row >= static_cast<long>(n_heads) * vdim,
               "attention_heads_mfma: a tensor is missing, a row is shorter than its heads, or a dtype is unknown");
  BC4G_REQUIRE(reinterpret_cast<uintptr_t>(q) % 16 == 0 && reinterpret_cast<uintptr_t>(k_cache) % 16 == 0 && reinterpret_cast<uintptr_t>(v_cache) % 16 == 0,
               "attention_heads_mfma: queries and caches must lie on 16-byte boundaries");
  if (n_seqs == 0 || most_rows == 0) return 0;
  const long tiles = (static_cast<long>(most_rows) * (n_heads / n_kv_heads) + kRowsAGroup - 1) / kRowsAGroup;
  BC4G_REQUIRE(tiles * n_kv_heads <= 2147483647L, "attention_heads_mfma: too many tiles");
  int shift = -1;
  for (int b = 0; b < 31; ++b)
    if (page_tokens == 1 << b) shift = b;
  const int wide_out = reinterpret_cast<uintptr_t>(out) % 8 == 0 && out_row % 4 == 0 ? 1 : 0;
  const HeadsArgs a{q, q_row, static_cast<const bf16_t*>(k_cache), static_cast<const bf16_t*>(v_cache), block_table, table_stride, seq_start,
                    seq_ctx, out, out_dtype, out_row, n_heads, n_kv_heads, dim, vdim, page_tokens, shift, window, static_cast<int>(tiles),
                    wide_out, scale, factor, sink};
  const dim3 grid(static_cast<unsigned>(tiles * n_kv_heads), n_seqs);
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (dim <= 32) launch_heads_values<1>(a, grid, s);
  else if (dim <= 64) launch_heads_values<2>(a, grid, s);
  else if (dim <= 128) launch_heads_values<4>(a, grid, s);
  else launch_heads_values<8>(a, grid, s);
  return check_launch("attention_heads_mfma");
}
