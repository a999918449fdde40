// Linear attention with a matrix memory per head, exponential input gates and a normaliser:
//
//   m_t = max(f_t + m_(t-1), i_t)                                                       m, S, n from zero
//   S_t = e^(f_t + m_(t-1) - m_t) S_(t-1) + e^(i_t - m_t) k_t v_t^T                     S [dim, vdim] per request and head
//   n_t = e^(f_t + m_(t-1) - m_t) n_(t-1) + e^(i_t - m_t) k_t                           n [dim]
//   o_t = S_t^T q_t / (max(|n_t . q_t|, e^(-m_t)) + 1e-6),  q scaled by a constant
//   out = o_t / rms(o_t) * weight * sigmoid(gate) * factor                               a head; rounded once, here
//
// with log gates i = cap tanh((zi + bi) / cap) and f = log sigmoid(cap tanh((zf + bf) / cap)), a number a head and row.
// Gates, m, S, n and all sums are float32; q, k, v, the gates' logits and the output gate are parts of one product's rows.
//
// As in decay_scan.hip a request's rows are walked in chunks of 32, a workgroup each, a thread keeping one column of S in
// registers (the workgroup has a thread for every column, so that a head's root mean square is taken where its values
// are made); the first wave also keeps n, its channels spread over the lanes.  A request of one chunk (a short portion) is
// one launch, from and into its slot; a step in which every request brings one row (decoding) is one launch of a kernel of
// its own, whose threads share a state's channels too, a few pieces of 16 bytes each.  Longer requests: the gates of all rows (m is a scan over pairs
// (A, B), m -> max(m + A, B)), every chunk from nothing (what it adds, the product of its decays), the states between the
// chunks, then every chunk again from its true state, writing outputs.
#include <math.h>

#include "api.h"
#include "common.h"

namespace bc4g {
namespace {

constexpr int kChunk = 32;       // rows of a request that one workgroup walks
constexpr int kStage = 16;       // rows whose q and k lie in LDS at a time
constexpr int kMaxV = 256;       // values a head
constexpr int kGateThreads = 1024;

struct MemoryArgs {
  const void *q, *k, *v, *gate, *zi, *zf;      // parts of rows `row` elements apart, all of one dtype
  long row;
  int dtype;
  const float *bi, *bf;                        // [heads]
  const float* weight;                         // [heads * vdim]
  float cap, q_scale, eps, factor;
  void* out;                                   // [T, heads * vdim], rows out_row apart
  int out_dtype;
  long out_row;
  float *S, *n, *m;                            // [slots, heads, dim, vdim], [slots, heads, dim], [slots, heads]
  float* gates;                                // [3][T][heads]: decay, input weight, m of every row (requests of several chunks)
  float *chunk_S, *chunk_n, *chunk_decay;      // [chunks, heads, dim, vdim], [chunks, heads, dim], [chunks, heads]
  const int32_t *seq_start, *seq_slots, *chunk_base;
  int n_rows, heads, dim, vdim;
};

__device__ inline float load_any(const void* p, int dtype, long idx) {
  return dtype == kF32 ? static_cast<const float*>(p)[idx] : to_float(static_cast<const bf16_t*>(p)[idx]);
}
__device__ inline float log_sigmoid(float z) { return -(fmaxf(-z, 0.f) + log1pf(expf(-fabsf(z)))); }

__device__ inline void log_gates(const MemoryArgs& a, long row, int head, float& i, float& f) {
  i = a.cap * tanhf((load_any(a.zi, a.dtype, row * a.row + head) + a.bi[head]) / a.cap);
  f = log_sigmoid(a.cap * tanhf((load_any(a.zf, a.dtype, row * a.row + head) + a.bf[head]) / a.cap));
}

// Along the wave's lanes: (A, B) becomes the composition of the lanes' maps m -> max(m + A, B) from lane 0 on.
__device__ inline void scan_maps(float& A, float& B, int lane) {
#pragma unroll
  for (int off = 1; off < kWave; off <<= 1) {
    const float a0 = __shfl_up(A, off, kWave), b0 = __shfl_up(B, off, kWave);
    if (lane >= off) {
      B = fmaxf(b0 + A, B);
      A = a0 + A;
    }
  }
}

// Every row's decay, input weight and m, for the requests of several chunks; a workgroup a (request, head).
__global__ __launch_bounds__(kGateThreads) void memory_gates_kernel(const MemoryArgs a) {
  __shared__ float wave_A[kGateThreads / kWave], wave_B[kGateThreads / kWave], last_m[kGateThreads / kWave];
  const int head = blockIdx.x, s = blockIdx.y, lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
  const long start = a.seq_start[s], end = a.seq_start[s + 1];
  if (end - start <= kChunk) return;
  const long slot = static_cast<long>(a.seq_slots[s]) * a.heads + head, per = static_cast<long>(a.n_rows) * a.heads;
  float m_in = a.m[slot];
  for (long r0 = start; r0 < end; r0 += kGateThreads) {
    const long row = r0 + threadIdx.x;
    const bool live = row < end;
    float i = 0.f, f = 0.f;
    if (live) log_gates(a, row, head, i, f);
    float A = live ? f : 0.f, B = live ? i : -INFINITY;      // (no row: the map that changes nothing)
    scan_maps(A, B, lane);
    if (lane == kWave - 1) wave_A[wave] = A, wave_B[wave] = B;
    __syncthreads();
    float m0 = m_in;                                          // m before this wave's first row
    for (int w = 0; w < wave; ++w) m0 = fmaxf(m0 + wave_A[w], wave_B[w]);
    const float m = fmaxf(m0 + A, B);
    if (lane == kWave - 1) last_m[wave] = m;
    __syncthreads();
    float before = __shfl_up(m, 1, kWave);                    // (the row before's own m, not another rounding of it)
    if (lane == 0) before = wave > 0 ? last_m[wave - 1] : m_in;
    if (live) {
      const long at = row * a.heads + head;
      a.gates[at] = expf(f + before - m);
      a.gates[per + at] = expf(i - m);
      a.gates[2 * per + at] = m;
    }
    m_in = last_m[kGateThreads / kWave - 1];                  // (rows that are not there carry m on)
    __syncthreads();
  }
  if (threadIdx.x == 0) a.m[slot] = m_in;
}

// kPass 0: the chunk from nothing -> chunk_S, chunk_n, chunk_decay.  kPass 1: the chunk from its true state -> out (and,
// for a request of one chunk, the slot).  Grid: (chunks of the longest request, S * heads); a thread a column of S.
template <int KD, int kPass>
__global__ __launch_bounds__(kMaxV) void memory_scan_kernel(const MemoryArgs a) {
  constexpr int NPL = (KD + kWave - 1) / kWave;      // channels of n a lane of the first wave keeps
  __shared__ float k_s[kStage][KD];                  // keys times their input weights
  __shared__ float q_s[kPass ? kStage : 1][KD];
  __shared__ float o_s[kPass ? kStage : 1][kPass ? kMaxV : 1];
  __shared__ float dec_s[kChunk], add_s[kChunk], top_s[kChunk], den_s[kStage];
  const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, n_waves = blockDim.x / kWave;
  const int chunk = blockIdx.x, s = blockIdx.y / a.heads, head = blockIdx.y % a.heads;
  const int dim = a.dim, vdim = a.vdim;
  const long start = a.seq_start[s], end = a.seq_start[s + 1];
  const int n_chunks = static_cast<int>((end - start + kChunk - 1) / kChunk);
  if (chunk >= n_chunks || (kPass == 0 && n_chunks < 2)) return;
  const long lo = start + static_cast<long>(chunk) * kChunk, hi = lo + kChunk < end ? lo + kChunk : end;
  const bool live = tid < vdim;
  const long slot = static_cast<long>(a.seq_slots[s]) * a.heads + head;
  const long from = n_chunks >= 2 ? static_cast<long>(a.chunk_base[s] + chunk) * a.heads + head : slot;
  const long per_state = static_cast<long>(dim) * vdim;

  if (wave == 0) {                                   // the chunk's gates, a row a lane
    const long row = lo + lane;
    const bool there = lane < kChunk && row < hi;
    float dec = 1.f, add = 0.f, m = 0.f;
    if (n_chunks >= 2) {
      if (there) {
        const long at = row * a.heads + head, per = static_cast<long>(a.n_rows) * a.heads;
        dec = a.gates[at], add = a.gates[per + at], m = a.gates[2 * per + at];
      }
    } else {
      float i = 0.f, f = 0.f;
      if (there) log_gates(a, row, head, i, f);
      const float m_in = a.m[slot];
      float A = there ? f : 0.f, B = there ? i : -INFINITY;
      scan_maps(A, B, lane);
      m = fmaxf(m_in + A, B);
      float before = __shfl_up(m, 1, kWave);
      if (lane == 0) before = m_in;
      dec = expf(f + before - m), add = expf(i - m);
      if (kPass && lane == kWave - 1) a.m[slot] = m;   // (nobody else reads this slot's m)
    }
    if (lane < kChunk) dec_s[lane] = dec, add_s[lane] = add, top_s[lane] = m;
  }

  float S[KD], n[NPL];
#pragma unroll
  for (int d = 0; d < KD; ++d) S[d] = 0.f;
#pragma unroll
  for (int i = 0; i < NPL; ++i) n[i] = 0.f;
  if (kPass) {
    const float* S0 = (n_chunks >= 2 ? a.chunk_S : a.S) + from * per_state + tid;
    const float* n0 = (n_chunks >= 2 ? a.chunk_n : a.n) + from * dim;
#pragma unroll
    for (int d = 0; d < KD; ++d) S[d] = (live && d < dim) ? S0[static_cast<long>(d) * vdim] : 0.f;
    if (wave == 0)
#pragma unroll
      for (int i = 0; i < NPL; ++i) n[i] = lane + i * kWave < dim ? n0[lane + i * kWave] : 0.f;
  }
  for (long r0 = lo; r0 < hi; r0 += kStage) {
    const int nr = static_cast<int>(hi - r0 < kStage ? hi - r0 : kStage), at0 = static_cast<int>(r0 - lo);
    __syncthreads();                                 // (the gates are written; the stage before has been read)
    // The rows lie in LDS KD wide, zeros beyond dim, so that the walk has no condition in it; four elements a thread asked
    // for together.
    for (int idx0 = tid; idx0 < nr * KD; idx0 += blockDim.x * 4) {
      float kk[4], qq[4];
#pragma unroll
      for (int b = 0; b < 4; ++b) {
        const int idx = idx0 + b * blockDim.x, r = idx / KD, d = idx % KD;
        const bool ok = r < nr && d < dim;
        const long at = (r0 + (ok ? r : 0)) * a.row + static_cast<long>(head) * dim + (ok ? d : 0);
        kk[b] = load_any(a.k, a.dtype, at);
        qq[b] = kPass ? load_any(a.q, a.dtype, at) : 0.f;
      }
#pragma unroll
      for (int b = 0; b < 4; ++b) {
        const int idx = idx0 + b * blockDim.x, r = idx / KD, d = idx % KD;
        if (r < nr) {
          k_s[r][d] = d < dim ? kk[b] * add_s[at0 + r] : 0.f;
          if (kPass) q_s[r][d] = d < dim ? qq[b] * a.q_scale : 0.f;
        }
      }
    }
    float vv[kStage];                                // this thread's column of the stage's values, asked for together
#pragma unroll
    for (int r = 0; r < kStage; ++r)
      vv[r] = (live && r < nr) ? load_any(a.v, a.dtype, (r0 + r) * a.row + static_cast<long>(head) * vdim + tid) : 0.f;
    __syncthreads();
    if (wave == 0) {                                 // the normaliser, and what every row's output is divided by
      float dot[kStage];
#pragma unroll
      for (int r = 0; r < kStage; ++r) {
        dot[r] = 0.f;
        if (r < nr) {
          const float dec = dec_s[at0 + r];
#pragma unroll
          for (int i = 0; i < NPL; ++i) {
            const int d = lane + i * kWave;
            const bool ok = d < KD;
            n[i] = fmaf(dec, n[i], ok ? k_s[r][ok ? d : 0] : 0.f);
            if (kPass) dot[r] = fmaf(n[i], ok ? q_s[r][ok ? d : 0] : 0.f, dot[r]);
          }
        }
      }
      if (kPass) {
#pragma unroll
        for (int r = 0; r < kStage; ++r) {
          const float total = wave_sum(dot[r]);
          if (lane == 0 && r < nr) den_s[r] = fmaxf(fabsf(total), expf(-top_s[at0 + r])) + 1e-6f;
        }
      }
    }
#pragma unroll
    for (int r = 0; r < kStage; ++r) {
      if (r >= nr) break;
      const float dec = dec_s[at0 + r];
      float o = 0.f;
#pragma unroll
      for (int d = 0; d < KD; ++d) {
        S[d] = fmaf(dec, S[d], k_s[r][d] * vv[r]);
        if (kPass) o = fmaf(S[d], q_s[r][d], o);
      }
      if (kPass) o_s[r][tid] = o;
    }
    if (kPass) {
      __syncthreads();
      for (int r = wave; r < nr; r += n_waves) {      // a wave a row: the head's root mean square, weight and gate
        const float den = den_s[r];
        float val[kMaxV / kWave], ss = 0.f;
#pragma unroll
        for (int i = 0; i < kMaxV / kWave; ++i) {
          const int c = lane + i * kWave;
          val[i] = c < vdim ? o_s[r][c] / den : 0.f;
          ss = fmaf(val[i], val[i], ss);
        }
        const float by = a.factor / sqrtf(wave_sum(ss) / static_cast<float>(vdim) + a.eps);
#pragma unroll
        for (int i = 0; i < kMaxV / kWave; ++i) {
          const int c = lane + i * kWave;
          if (c >= vdim) break;
          const long col = static_cast<long>(head) * vdim + c;
          const float g = load_any(a.gate, a.dtype, (r0 + r) * a.row + col);
          const float y = val[i] * by * a.weight[col] / (1.0f + expf(-g));
          const long to = (r0 + r) * a.out_row + col;
          if (a.out_dtype == kF32) static_cast<float*>(a.out)[to] = y;
          else static_cast<bf16_t*>(a.out)[to] = from_float<bf16_t>(y);
        }
      }
    }
  }
  if (kPass == 1 && n_chunks >= 2) return;           // (the pass between the chunks has left the slot's state)
  float* S1 = (kPass == 0 ? a.chunk_S : a.S) + from * per_state + tid;
  float* n1 = (kPass == 0 ? a.chunk_n : a.n) + from * dim;
  if (live) {
#pragma unroll
    for (int d = 0; d < KD; ++d)
      if (d < dim) S1[static_cast<long>(d) * vdim] = S[d];
  }
  if (wave == 0) {
#pragma unroll
    for (int i = 0; i < NPL; ++i)
      if (lane + i * kWave < dim) n1[lane + i * kWave] = n[i];
  }
  if (kPass == 0 && tid == 0) {
    float prod = 1.f;
    for (int r = 0; r < static_cast<int>(hi - lo); ++r) prod *= dec_s[r];
    a.chunk_decay[from] = prod;
  }
}

// Between the passes: a thread takes one element of S (or, behind those, of n) of one (request, head) with two chunks or
// more, replaces every chunk's sum by the state before the chunk and leaves the state after the last one in the slot.
__global__ void memory_between_kernel(const MemoryArgs a) {
  const int s = blockIdx.y / a.heads, head = blockIdx.y % a.heads;
  const int n_chunks = (a.seq_start[s + 1] - a.seq_start[s] + kChunk - 1) / kChunk;
  if (n_chunks < 2) return;
  const long per_S = static_cast<long>(a.dim) * a.vdim;
  long e = blockIdx.x * static_cast<long>(blockDim.x) + threadIdx.x;
  if (e >= per_S + a.dim) return;
  const bool is_n = e >= per_S;
  const long per = is_n ? a.dim : per_S;
  if (is_n) e -= per_S;
  float* slot = (is_n ? a.n : a.S) + (static_cast<long>(a.seq_slots[s]) * a.heads + head) * per + e;
  float* chunks = (is_n ? a.chunk_n : a.chunk_S) + e;
  float st = *slot;
  const long id0 = a.chunk_base[s];
  for (int c0 = 0; c0 < n_chunks; c0 += 8) {          // (eight chunks' numbers asked for together)
    float add[8], dec[8];
#pragma unroll
    for (int b = 0; b < 8; ++b) {
      const bool ok = c0 + b < n_chunks;
      const long id = (id0 + (ok ? c0 + b : 0)) * a.heads + head;
      add[b] = ok ? chunks[id * per] : 0.f;
      dec[b] = ok ? a.chunk_decay[id] : 1.f;
    }
#pragma unroll
    for (int b = 0; b < 8; ++b) {
      if (c0 + b < n_chunks) {
        chunks[((id0 + c0 + b) * a.heads + head) * per] = st;
        st = fmaf(dec[b], st, add[b]);
      }
    }
  }
  *slot = st;
}

// A step of one row a request: a workgroup a (request, head), its threads in groups of whole rows of S -- thread t takes VEC
// neighbouring columns and every n_groups-th channel --, so that all of a state's memory is asked for at once.
constexpr int kStepThreads = 512;
template <int VEC>
__global__ __launch_bounds__(kStepThreads) void memory_step_kernel(const MemoryArgs a) {
  __shared__ float part_s[kStepThreads * VEC];
  __shared__ float red_s[kStepThreads / kWave];
  __shared__ float scratch[16];
  constexpr int kAhead = 8;
  const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave;
  const int s = blockIdx.x / a.heads, head = blockIdx.x % a.heads, dim = a.dim, vdim = a.vdim;
  const long row = a.seq_start[s], slot = static_cast<long>(a.seq_slots[s]) * a.heads + head;
  const int cols = vdim / VEC, groups = kStepThreads / cols, group = tid / cols, c0 = (tid % cols) * VEC;
  const bool mine = group < groups;
  float* S = a.S + slot * dim * vdim;
  const long at_k = row * a.row + static_cast<long>(head) * dim, at_v = row * a.row + static_cast<long>(head) * vdim;

  // Pieces of the state and the keys and queries that go with them; the first are on their way while the gates are made.
  float have[kAhead][VEC], kk[kAhead], qq[kAhead];
  auto fetch = [&](int d0) {
#pragma unroll
    for (int b = 0; b < kAhead; ++b) {
      const int d = d0 + b * groups;
      const bool ok = mine && d < dim;
      const float* from = S + static_cast<long>(ok ? d : 0) * vdim + (ok ? c0 : 0);
      if constexpr (VEC == 4) {
        const float4 x = *reinterpret_cast<const float4*>(from);
        have[b][0] = x.x, have[b][1] = x.y, have[b][2] = x.z, have[b][3] = x.w;
      } else {
        have[b][0] = *from;
      }
      kk[b] = load_any(a.k, a.dtype, at_k + (ok ? d : 0));
      qq[b] = load_any(a.q, a.dtype, at_k + (ok ? d : 0));
    }
  };
  fetch(group);
  float v[VEC];
#pragma unroll
  for (int e = 0; e < VEC; ++e) v[e] = mine ? load_any(a.v, a.dtype, at_v + c0 + e) : 0.f;
  float i, f;
  log_gates(a, row, head, i, f);
  const float m_in = a.m[slot], m = fmaxf(f + m_in, i);
  const float dec = expf(f + m_in - m), add = expf(i - m);

  float dot = 0.f;
  for (int d = tid; d < dim; d += kStepThreads) {
    const float nd = fmaf(dec, a.n[slot * dim + d], add * load_any(a.k, a.dtype, at_k + d));
    a.n[slot * dim + d] = nd;
    dot = fmaf(nd, load_any(a.q, a.dtype, at_k + d) * a.q_scale, dot);
  }
  dot = wave_sum(dot);
  if (lane == 0) red_s[wave] = dot;

  float o[VEC];
#pragma unroll
  for (int e = 0; e < VEC; ++e) o[e] = 0.f;
  for (int d0 = group; d0 < dim; d0 += groups * kAhead) {
    if (d0 != group) fetch(d0);
#pragma unroll
    for (int b = 0; b < kAhead; ++b) {
      const int d = d0 + b * groups;
      if (!mine || d >= dim) continue;
      const float k = add * kk[b], q = a.q_scale * qq[b];
      float now[VEC];
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        now[e] = fmaf(dec, have[b][e], k * v[e]);
        o[e] = fmaf(now[e], q, o[e]);
      }
      float* to = S + static_cast<long>(d) * vdim + c0;
      if constexpr (VEC == 4) *reinterpret_cast<float4*>(to) = make_float4(now[0], now[1], now[2], now[3]);
      else to[0] = now[0];
    }
  }
#pragma unroll
  for (int e = 0; e < VEC; ++e)
    if (mine) part_s[group * vdim + c0 + e] = o[e];
  __syncthreads();
  if (tid == 0) a.m[slot] = m;                        // (every thread has read the old one)
  float total = 0.f;
  for (int w = 0; w < kStepThreads / kWave; ++w) total += red_s[w];
  const float den = fmaxf(fabsf(total), expf(-m)) + 1e-6f;
  float val = 0.f;
  if (tid < vdim) {
    for (int g = 0; g < groups; ++g) val += part_s[g * vdim + tid];
    val /= den;
  }
  const float by = a.factor / sqrtf(block_sum(val * val, scratch) / static_cast<float>(vdim) + a.eps);
  if (tid < vdim) {
    const long col = static_cast<long>(head) * vdim + tid;
    const float y = val * by * a.weight[col] / (1.0f + expf(-load_any(a.gate, a.dtype, row * a.row + col)));
    if (a.out_dtype == kF32) static_cast<float*>(a.out)[row * a.out_row + col] = y;
    else static_cast<bf16_t*>(a.out)[row * a.out_row + col] = from_float<bf16_t>(y);
  }
}

template <int KD>
void launch_memory(const MemoryArgs& a, int n_seqs, int most_chunks, hipStream_t s) {
  dim3 grid(most_chunks, n_seqs * a.heads), block(ceil_div(a.vdim, kWave) * kWave);
  if (most_chunks >= 2) {
    memory_gates_kernel<<<dim3(a.heads, n_seqs), kGateThreads, 0, s>>>(a);
    memory_scan_kernel<KD, 0><<<grid, block, 0, s>>>(a);
    memory_between_kernel<<<dim3(ceil_div(static_cast<long>(a.dim) * (a.vdim + 1), 256), n_seqs * a.heads), 256, 0, s>>>(a);
  }
  memory_scan_kernel<KD, 1><<<grid, block, 0, s>>>(a);
}

}  // namespace
}  // namespace bc4g

using namespace bc4g;

extern "C" int bc4g_matrix_memory(const void* q, const void* k, const void* v, const void* gate, const void* zi, const void* zf,
                                  int dtype, long row, const float* bi, const float* bf, float cap, float q_scale,
                                  const float* weight, float eps, float factor, void* out, int out_dtype, long out_row, float* S,
                                  float* n, float* m, float* gates, float* chunk_S, float* chunk_n, float* chunk_decay,
                                  const int32_t* seq_start, const int32_t* seq_slots, const int32_t* chunk_base, int n_rows,
                                  int n_seqs, int most_rows, int heads, int dim, int vdim, void* stream) {
  BC4G_REQUIRE(n_rows >= 0 && n_seqs >= 0 && most_rows >= 0 && heads > 0 && dim > 0 && dim <= 256 && vdim > 0 && vdim <= kMaxV,
               "matrix_memory: bad sizes T=%d S=%d heads=%d dim=%d (at most 256) vdim=%d (at most %d)", n_rows, n_seqs, heads, dim,
               vdim, kMaxV);
  BC4G_REQUIRE(static_cast<long>(n_seqs) * heads <= 65535, "matrix_memory: %d requests x %d heads are beyond the grid limit", n_seqs, heads);
  BC4G_REQUIRE(q && k && v && gate && zi && zf && bi && bf && weight && out && S && n && m && seq_start && seq_slots && cap > 0.f,
               "matrix_memory: a tensor is missing, or the gates' cap %g is not positive", static_cast<double>(cap));
  BC4G_REQUIRE((dtype == kF32 || dtype == kBF16) && (out_dtype == kF32 || out_dtype == kBF16) &&
               row >= static_cast<long>(heads) * (dim > vdim ? dim : vdim) && out_row >= static_cast<long>(heads) * vdim,
               "matrix_memory: a row is shorter than its heads, or a dtype is unknown");
  if (n_rows == 0 || n_seqs == 0 || most_rows == 0) return 0;
  const int most_chunks = ceil_div(most_rows, kChunk);
  BC4G_REQUIRE(most_chunks < 2 || (gates && chunk_S && chunk_n && chunk_decay && chunk_base),
               "matrix_memory: requests of several chunks need scratch memory");
  const MemoryArgs a{q, k, v, gate, zi, zf, row, dtype, bi, bf, weight, cap, q_scale, eps, factor, out, out_dtype, out_row,
                     S, n, m, gates, chunk_S, chunk_n, chunk_decay, seq_start, seq_slots, chunk_base, n_rows, heads, dim, vdim};
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (most_rows == 1) {
    if (vdim % 4 == 0 && reinterpret_cast<uintptr_t>(S) % 16 == 0) memory_step_kernel<4><<<n_seqs * heads, kStepThreads, 0, s>>>(a);
    else memory_step_kernel<1><<<n_seqs * heads, kStepThreads, 0, s>>>(a);
    return check_launch("matrix_memory");
  }
  if (dim <= 16) launch_memory<16>(a, n_seqs, most_chunks, s);
  else if (dim <= 32) launch_memory<32>(a, n_seqs, most_chunks, s);
  else if (dim <= 64) launch_memory<64>(a, n_seqs, most_chunks, s);
  else if (dim <= 128) launch_memory<128>(a, n_seqs, most_chunks, s);
  else launch_memory<256>(a, n_seqs, most_chunks, s);
  return check_launch("matrix_memory");
}
