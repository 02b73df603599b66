// Gated linear attention: a matrix-valued recurrent state per head,
//   S_t = diag(a_t) S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t,
// with a decay a_t in (0, 1) per key channel.  Two relatives go through the same kernels:
//   bonus      o_t = (S_(t-1) + diag(u) k_t v_t^T)^T q_t: the current token through a learned vector u
//   memory     S_t = keep_t S_(t-1) + take_t k_t v_t^T,  n_t = keep_t n_(t-1) + take_t k_t, with one number
//              keep_t and take_t per head from exponential gates and a running maximum (below)
// The state [D, E] per head lives in float32 in
// a slot per request and is carried from step to step; everything here is float32.  gfx950.
//
// Three kernels: the decays from their low-rank projection; the scan over the tokens of every
// request of the step (prompts' portions and single decoded tokens alike); the output
// (norm over each head's values, gate, rounding to the compute dtype).
#include <type_traits>

#include "common.h"

extern "C" const char* llmlab_last_error() { return g_llmlab_error; }

constexpr int SLICE = 16;      // key channels of the state that one thread keeps in registers

// ---------------------------------------------------------------------- decays
// a[r, c] = sigmoid(z)^(1 / tau), z = bias[c] + sum_j w2[c, j] * low[r, j]  (c over heads * D
// key channels, j over the rank of the projection).  sigmoid(z)^(1/tau) = exp(-softplus(-z) / tau),
// with softplus(u) = max(u, 0) + log1p(exp(-|u|)), so that neither end overflows.
// kind 1 (DECAY_DOUBLE_EXP): a[r, c] = exp(-exp(z)), z = bias[c] + sum_j w2[c, j] * tanh(low[r, j]).
// as_log: the decay's logarithm to the base 2 instead, at least LOG_FLOOR (what the chunked scan on the
// matrix cores takes; a decay of 2^-60 leaves nothing of a state in 32 bits).
constexpr int DECAY_SIGMOID = 0, DECAY_DOUBLE_EXP = 1;
constexpr float LOG2_E = 1.4426950408889634f, LOG_FLOOR = -60.f;
__device__ __forceinline__ float log_decay_of(float z, int kind, float inv_tau) {
  if (kind == DECAY_DOUBLE_EXP) return -expf(z);
  const float u = -z;
  return -(fmaxf(u, 0.f) + log1pf(expf(-fabsf(u)))) * inv_tau;
}
__device__ __forceinline__ float decay_of(float z, int kind, float inv_tau) { return expf(log_decay_of(z, kind, inv_tau)); }
__global__ __launch_bounds__(256) void gla_decay_kernel(const float* __restrict__ low, int ld, int rank,
                                                        const float* __restrict__ w2, const float* __restrict__ bias,
                                                        int kind, float inv_tau, float* __restrict__ decay, int channels,
                                                        int as_log) {
  extern __shared__ float s_low[];
  const int r = blockIdx.x;
  const float* t = low + (size_t)r * ld;
  for (int j = threadIdx.x; j < rank; j += blockDim.x) s_low[j] = kind == DECAY_DOUBLE_EXP ? tanhf(t[j]) : t[j];
  __syncthreads();
  for (int c = threadIdx.x; c < channels; c += blockDim.x) {
    float z = bias ? bias[c] : 0.f;
    const float* w = w2 + (size_t)c * rank;
    if ((rank & 3) == 0) {                       // (a row of the second factor 16 bytes a load, all on their way together)
      for (int j = 0; j < rank; j += 4) {
        const floatx4 w4 = *(const floatx4*)(w + j);
        z = fmaf(w4[0], s_low[j], z);
        z = fmaf(w4[1], s_low[j + 1], z);
        z = fmaf(w4[2], s_low[j + 2], z);
        z = fmaf(w4[3], s_low[j + 3], z);
      }
    } else {
      for (int j = 0; j < rank; ++j) z = fmaf(w[j], s_low[j], z);
    }
    const float lg = log_decay_of(z, kind, inv_tau);
    decay[(size_t)r * channels + c] = as_log ? fmaxf(lg * LOG2_E, LOG_FLOOR) : expf(lg);
  }
}

extern "C" int llmlab_gla_decay(const float* low, int ld, int rows, int rank, const float* w2, const float* bias,
                                int kind, float tau, float* decay, int channels, int as_log, hipStream_t stream) {
  LLMLAB_REQUIRE(rows >= 0 && rank > 0 && rank <= 8192 && channels > 0 && ld >= rank && tau > 0.f &&
                     (kind == DECAY_SIGMOID || kind == DECAY_DOUBLE_EXP),
                 "gla_decay: bad sizes rows=%d rank=%d channels=%d ld=%d kind=%d tau=%g", rows, rank, channels, ld, kind,
                 (double)tau);
  if (rows == 0) return 0;
  hipLaunchKernelGGL(gla_decay_kernel, dim3(rows), dim3(256), rank * sizeof(float), stream, low, ld, rank, w2, bias, kind,
                     1.0f / tau, decay, channels, as_log);
  LLMLAB_LAUNCH_CHECK("gla_decay");
  return 0;
}

// ---------------------------------------------------------- gates of a matrix memory
// Per head and row the log gates i = cap * tanh((proj_i + bias_i) / cap) and f = logsigmoid(cap *
// tanh((proj_f + bias_f) / cap)), the running maximum m_t = max(f_t + m_(t-1), i_t) from the slot's (0 at
// a sequence's start), and what the recurrence multiplies by: keep = exp(f_t + m_(t-1) - m_t), take =
// exp(i_t - m_t).  All float32.  Block (request, head): the rows MEMORY_TILE at a time, a thread a
// row; the maxima of a tile by a scan over (sum of f, maximum so far) pairs, (F1, M1) then (F2, M2) =
// (F1 + F2, max(M1 + F2, M2)).  Whatever rounding the scan adds to an m, keep and take of all rows
// are taken from the same m's, so the state stays exact in them.
constexpr int MEMORY_TILE = 1024;
__global__ __launch_bounds__(MEMORY_TILE) void memory_gates_kernel(
    const float* __restrict__ proj, int ld, int off_i, int off_f, const float* __restrict__ bias_i,
    const float* __restrict__ bias_f, float cap, int n_heads, float* __restrict__ max_state, const int* __restrict__ q_start,
    const int* __restrict__ req_rows, float* __restrict__ keep, float* __restrict__ take, float* __restrict__ maxima,
    int as_log) {
  __shared__ float s_f[MEMORY_TILE / 64], s_m[MEMORY_TILE / 64], s_max[MEMORY_TILE + 1];
  const int b = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int first = q_start[b], last = q_start[b + 1];
  if (first >= last) return;
  float* slot = max_state + (size_t)req_rows[b] * n_heads + h;
  float carry = *slot;
  const float bi = bias_i ? bias_i[h] : 0.f, bf = bias_f ? bias_f[h] : 0.f;
  for (int t0 = first; t0 < last; t0 += MEMORY_TILE) {
    const int t = t0 + (int)threadIdx.x;
    const bool in = t < last;
    float i = -__builtin_huge_valf(), f = 0.f;      // (rows past the end leave the maximum as it is)
    if (in) {
      const float* row = proj + (size_t)t * ld;
      i = cap * tanhf((row[off_i + h] + bi) / cap);
      const float z = cap * tanhf((row[off_f + h] + bf) / cap);
      f = -(fmaxf(-z, 0.f) + log1pf(expf(-fabsf(z))));
    }
    float F = f, M = i;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const float F1 = __shfl_up(F, off, WAVE), M1 = __shfl_up(M, off, WAVE);
      if (lane >= off) {
        M = fmaxf(M1 + F, M);
        F = F1 + F;
      }
    }
    if (lane == 63) {
      s_f[wave] = F;
      s_m[wave] = M;
    }
    if (threadIdx.x == 0) s_max[0] = carry;
    __syncthreads();
    float m0 = carry;                               // the maximum before this wave's rows
    for (int w = 0; w < wave; ++w) m0 = fmaxf(s_f[w] + m0, s_m[w]);
    const float m = fmaxf(F + m0, M);
    s_max[threadIdx.x + 1] = m;
    __syncthreads();
    if (in) {
      const size_t at = (size_t)t * n_heads + h;
      const float lg = f + s_max[threadIdx.x] - m;
      keep[at] = as_log ? fmaxf(lg * LOG2_E, LOG_FLOOR) : expf(lg);      // (as for the decays)
      take[at] = expf(i - m);
      maxima[at] = m;
    }
    carry = s_max[MEMORY_TILE];
    __syncthreads();
  }
  if (threadIdx.x == 0) *slot = carry;
}

extern "C" int llmlab_memory_gates(const float* proj, int ld, int off_i, int off_f, const float* bias_i, const float* bias_f,
                                   float cap, int n_heads, float* max_state, const int* q_start, const int* req_rows,
                                   int n_reqs, float* keep, float* take, float* maxima, int as_log, hipStream_t stream) {
  LLMLAB_REQUIRE(n_reqs >= 0 && n_heads > 0 && n_heads <= 65535 && cap > 0.f && off_i >= 0 && off_f >= 0 &&
                     ld >= off_i + n_heads && ld >= off_f + n_heads,
                 "memory_gates: bad sizes requests=%d heads=%d cap=%g ld=%d", n_reqs, n_heads, (double)cap, ld);
  LLMLAB_REQUIRE(proj && max_state && q_start && req_rows && keep && take && maxima, "memory_gates: an operand is missing");
  if (n_reqs == 0) return 0;
  hipLaunchKernelGGL(memory_gates_kernel, dim3(n_reqs, n_heads), dim3(MEMORY_TILE), 0, stream, proj, ld, off_i, off_f, bias_i,
                     bias_f, cap, n_heads, max_state, q_start, req_rows, keep, take, maxima, as_log);
  LLMLAB_LAUNCH_CHECK("memory_gates");
  return 0;
}

// ------------------------------------------------------------------------ scan
// Thread (s, e) of a block keeps the SLICE rows s * SLICE .. of column e of one head's state in
// registers, walks a run of rows in order, and leaves its part of o_t in parts[row, h, s, e];
// the output kernel adds the parts of the slices.  Threads never talk to each other, so a
// token costs no barrier; the loads of a token do not depend on the state, so they run
// ahead of the sums.
//
// WHOLE: a block takes all the rows that request blockIdx.x brings to the step: the state
// comes from the request's slot and goes back there.  That is the kernel of decode steps
// and of short portions.
//
// Long portions are cut into chunks of `chunk` rows that run side by side, in three passes
// (the recurrence is linear in the state: S_end = P * S_start + L with P the product of the
// chunk's decays and L the state the chunk builds from zero):
//   LOCAL  per chunk: L and P, from a zero state, no outputs;
//   carry  per request, chunk after chunk: S_start[c], and the request's slot at the end;
//   FINISH per chunk: the rows again from S_start[c], now with outputs.
// All of it in float32; the result differs from the row-by-row recurrence by rounding only.
enum { SCAN_WHOLE = 0, SCAN_LOCAL = 1, SCAN_FINISH = 2 };
// KIND: DECAY and BONUS take a decay per key channel (and the bonus u [heads, D]); MEMORY one
// number keep_t and one take_t per head.  MEMORY's normaliser n (key channels only, no values) is
// the business of one more block per head (blockIdx.z past the columns): lane c < SLICE of slice s
// keeps n[d0 + c] and leaves the slice's part of n_t . q_t in norm_parts[row, h, s].
enum { KIND_DECAY = 0, KIND_BONUS = 1, KIND_MEMORY = 2 };

struct ScanArgs {
  const float* proj; int ld, off_q, off_k, off_v;
  const float* decay; float q_scale; int n_heads, D, E, cols, slices;
  float* state; const int* q_start; const int* req_rows; float* parts;
  int n_reqs, chunk; float* chunk_state; float* chunk_decay;      // [chunks, heads, D, E] and [chunks, heads, D]
  const float* bonus;                                              // BONUS: u [heads, D]
  const float* keep; const float* take;                            // MEMORY: [rows, heads]
  float* norm_state; float* norm_parts; float* chunk_norm;         // MEMORY: [slots, heads, D], [rows, heads, slices], [chunks, heads, D]
};

// Which request and which rows the chunk `index` of the step covers (chunks are counted
// request after request); false if the step has fewer chunks.
__device__ __forceinline__ bool find_chunk(const ScanArgs& a, int index, int& first, int& last) {
  int before = 0;
  for (int b = 0; b < a.n_reqs; ++b) {
    const int lo = a.q_start[b], hi = a.q_start[b + 1];
    const int n = (hi - lo + a.chunk - 1) / a.chunk;
    if (index < before + n) {
      first = lo + (index - before) * a.chunk;
      last = first + a.chunk < hi ? first + a.chunk : hi;
      return true;
    }
    before += n;
  }
  return false;
}

// The normaliser of one head over the rows [first, last): see KIND_MEMORY above.
template <int MODE>
__device__ __forceinline__ void scan_normaliser(const ScanArgs& a, int h, int first, int last) {
  const int c = threadIdx.x % a.cols, s = threadIdx.x / a.cols;
  const int D = a.D, d = s * SLICE + c;
  const bool mine = c < SLICE && s < a.slices && d < D;
  if (a.cols % SLICE != 0) {      // (a slice's lanes are no whole groups of 16 then: one lane a slice walks all its channels)
    if (c != 0 || s >= a.slices) return;
    float* st = (MODE == SCAN_WHOLE ? a.norm_state + ((size_t)a.req_rows[blockIdx.x] * a.n_heads + h) * D
                                    : a.chunk_norm + ((size_t)blockIdx.x * a.n_heads + h) * D) + s * SLICE;
    const int n = D - s * SLICE < SLICE ? D - s * SLICE : SLICE;
    float N[SLICE];
    for (int i = 0; i < SLICE; ++i) N[i] = (MODE != SCAN_LOCAL && i < n) ? st[i] : 0.f;
    for (int t = first; t < last; ++t) {
      const float* row = a.proj + (size_t)t * a.ld + h * D + s * SLICE;
      const float keep = a.keep[(size_t)t * a.n_heads + h], take = a.take[(size_t)t * a.n_heads + h];
      float acc = 0.f;
#pragma unroll
      for (int i = 0; i < SLICE; ++i) {
        N[i] = fmaf(keep, N[i], i < n ? take * row[a.off_k + i] : 0.f);
        if (MODE != SCAN_LOCAL) acc = fmaf(N[i], i < n ? row[a.off_q + i] : 0.f, acc);
      }
      if (MODE != SCAN_LOCAL) a.norm_parts[((size_t)t * a.n_heads + h) * a.slices + s] = acc * a.q_scale;
    }
    if (MODE == SCAN_FINISH) return;
    for (int i = 0; i < n; ++i) st[i] = N[i];
    return;
  }
  float* st = MODE == SCAN_WHOLE ? a.norm_state + ((size_t)a.req_rows[blockIdx.x] * a.n_heads + h) * D + d
                                 : a.chunk_norm + ((size_t)blockIdx.x * a.n_heads + h) * D + d;
  if (c >= SLICE || s >= a.slices) return;      // (whole quarters of a wave leave or stay: the sum below is over 16 lanes)
  float N = (MODE != SCAN_LOCAL && mine) ? *st : 0.f;
  struct Row { float keep, take, k, q; } r0, r1;
  auto fetch = [&](Row& r, int t) {
    const float* row = a.proj + (size_t)t * a.ld + h * D + d;
    r.keep = a.keep[(size_t)t * a.n_heads + h];
    r.take = a.take[(size_t)t * a.n_heads + h];
    r.k = mine ? row[a.off_k] : 0.f;
    if (MODE != SCAN_LOCAL) r.q = mine ? row[a.off_q] : 0.f;
  };
  auto step = [&](const Row& r, int t) {
    N = fmaf(r.keep, N, r.take * r.k);
    if (MODE == SCAN_LOCAL) return;
    float x = N * r.q;
#pragma unroll
    for (int off = 8; off > 0; off >>= 1) x += __shfl_xor(x, off, SLICE);
    if (c == 0) a.norm_parts[((size_t)t * a.n_heads + h) * a.slices + s] = x * a.q_scale;
  };
  if (first < last) fetch(r0, first);
  for (int t = first; t < last; t += 2) {
    if (t + 1 < last) fetch(r1, t + 1);
    step(r0, t);
    if (t + 1 < last) {
      if (t + 2 < last) fetch(r0, t + 2);
      step(r1, t + 1);
    }
  }
  if (MODE != SCAN_FINISH && mine) *st = N;
}

template <int MODE, int KIND, bool UNIFORM, int THREADS>
__global__ __launch_bounds__(THREADS) void gla_scan_kernel(ScanArgs a) {
  const int h = blockIdx.y;
  const int e = blockIdx.z * a.cols + (int)(threadIdx.x % a.cols);
  // UNIFORM: a wave lies within one slice (cols a multiple of 64), so the slice's decays,
  // keys and queries are the same for all its lanes and can come through the scalar unit
  const int s = UNIFORM ? __builtin_amdgcn_readfirstlane((int)(threadIdx.x / a.cols)) : (int)(threadIdx.x / a.cols);
  int first, last;
  if (MODE == SCAN_WHOLE) {
    first = a.q_start[blockIdx.x];
    last = a.q_start[blockIdx.x + 1];
  } else if (!find_chunk(a, blockIdx.x, first, last)) {
    return;
  }
  if (KIND == KIND_MEMORY && (int)blockIdx.z * a.cols >= a.E) {
    scan_normaliser<MODE>(a, h, first, last);
    return;
  }
  if (e >= a.E || s >= a.slices) return;
  const int D = a.D, E = a.E, d0 = s * SLICE;
  float S[SLICE], P[SLICE];
  float U[KIND == KIND_BONUS ? SLICE : 1];
  if (KIND == KIND_BONUS) {
#pragma unroll
    for (int i = 0; i < SLICE; ++i) U[i] = d0 + i < D ? a.bonus[h * D + d0 + i] : 0.f;
  }
  float* st = MODE == SCAN_WHOLE ? a.state + (((size_t)a.req_rows[blockIdx.x] * a.n_heads + h) * D + d0) * E + e
                                 : a.chunk_state + (((size_t)blockIdx.x * a.n_heads + h) * D + d0) * E + e;
#pragma unroll
  for (int i = 0; i < SLICE; ++i) {
    S[i] = (MODE != SCAN_LOCAL && d0 + i < D) ? st[(size_t)i * E] : 0.f;
    P[i] = 1.f;
  }
  // A row's decays, keys, queries and value are asked for one row ahead, so that their way
  // from memory overlaps the sums of the row before; two sets of registers take turns, so
  // nothing is copied.
  const bool whole = d0 + SLICE <= D;
  struct Row {
    float a[KIND == KIND_MEMORY ? 1 : SLICE], k[SLICE], q[SLICE], v;
  };
  auto fetch = [&](Row& r, int t) {
    const float* row = a.proj + (size_t)t * a.ld;
    const float* qp = row + a.off_q + h * D + d0;
    const float* kp = row + a.off_k + h * D + d0;
    const float* ap = KIND == KIND_MEMORY ? a.keep : a.decay + ((size_t)t * a.n_heads + h) * D + d0;
    r.v = row[a.off_v + h * E + e];
    if (KIND == KIND_MEMORY) {
      r.a[0] = a.keep[(size_t)t * a.n_heads + h];
      r.v *= a.take[(size_t)t * a.n_heads + h];
    }
#pragma unroll
    for (int i = 0; i < SLICE; ++i) {
      const bool in = whole || d0 + i < D;
      if (KIND != KIND_MEMORY) r.a[i] = in ? ap[i] : 1.f;
      r.k[i] = in ? kp[i] : 0.f;
      if (MODE != SCAN_LOCAL) r.q[i] = in ? qp[i] : 0.f;
    }
  };
  auto take = [&](const Row& r, int t) {
    float acc = 0.f;
#pragma unroll
    for (int i = 0; i < SLICE; ++i) {
      const float decay = r.a[KIND == KIND_MEMORY ? 0 : i], kv = r.k[i] * r.v;
      if (KIND == KIND_BONUS && MODE != SCAN_LOCAL) acc = fmaf(fmaf(U[i], kv, S[i]), r.q[i], acc);
      S[i] = fmaf(decay, S[i], kv);
      if (MODE == SCAN_LOCAL) P[i] *= decay;
      else if (KIND != KIND_BONUS) acc = fmaf(S[i], r.q[i], acc);
    }
    if (MODE != SCAN_LOCAL) a.parts[(((size_t)t * a.n_heads + h) * a.slices + s) * E + e] = acc * a.q_scale;
  };
  Row r0, r1;
  if (first < last) fetch(r0, first);
  for (int t = first; t < last; t += 2) {
    if (t + 1 < last) fetch(r1, t + 1);
    take(r0, t);
    if (t + 1 < last) {
      if (t + 2 < last) fetch(r0, t + 2);
      take(r1, t + 1);
    }
  }
  if (MODE == SCAN_FINISH) return;
#pragma unroll
  for (int i = 0; i < SLICE; ++i)
    if (d0 + i < D) st[(size_t)i * E] = S[i];
  if (MODE == SCAN_LOCAL && e == 0) {
    float* pd = a.chunk_decay + ((size_t)blockIdx.x * a.n_heads + h) * D + d0;
#pragma unroll
    for (int i = 0; i < SLICE; ++i)
      if (d0 + i < D) pd[i] = P[i];
  }
}

// One thread per element (h, d, e) of a request's state, chunk after chunk:
// chunk_state[c] <- the state before chunk c; the slot <- the state after the last chunk.  The numbers of
// CARRY_AHEAD chunks are asked for together.
constexpr int CARRY_AHEAD = 8;
__global__ __launch_bounds__(256) void gla_carry_kernel(ScanArgs a) {
  const int b = blockIdx.y;
  const size_t per = (size_t)a.n_heads * a.D * a.E;
  size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= per) {              // (behind the states' numbers the normalisers', if there are any)
    i -= per;
    const size_t hd_all = (size_t)a.n_heads * a.D;
    if (!a.norm_state || i >= hd_all) return;
    int c = 0;
    for (int r = 0; r < b; ++r) c += (a.q_start[r + 1] - a.q_start[r] + a.chunk - 1) / a.chunk;
    const int last = c + (a.q_start[b + 1] - a.q_start[b] + a.chunk - 1) / a.chunk;
    float* slot = a.norm_state + (size_t)a.req_rows[b] * hd_all + i;
    float N = *slot;
    for (; c < last; c += CARRY_AHEAD) {
      float built[CARRY_AHEAD], decay[CARRY_AHEAD];
#pragma unroll
      for (int x = 0; x < CARRY_AHEAD; ++x) {
        const size_t at = (size_t)(c + x < last ? c + x : last - 1) * hd_all + i;
        built[x] = a.chunk_norm[at];
        decay[x] = a.chunk_decay[at];
      }
#pragma unroll
      for (int x = 0; x < CARRY_AHEAD; ++x)
        if (c + x < last) {
          a.chunk_norm[(size_t)(c + x) * hd_all + i] = N;
          N = fmaf(decay[x], N, built[x]);
        }
    }
    *slot = N;
    return;
  }
  int before = 0;
  for (int r = 0; r < b; ++r) before += (a.q_start[r + 1] - a.q_start[r] + a.chunk - 1) / a.chunk;
  const int n = (a.q_start[b + 1] - a.q_start[b] + a.chunk - 1) / a.chunk;
  float* slot = a.state + (size_t)a.req_rows[b] * per + i;
  float S = *slot;
  const size_t hd = i / a.E;
  for (int c = before; c < before + n; c += CARRY_AHEAD) {
    float built[CARRY_AHEAD], decay[CARRY_AHEAD];
#pragma unroll
    for (int x = 0; x < CARRY_AHEAD; ++x) {      // (past the last: the last again, dropped)
      const size_t at = (size_t)(c + x < before + n ? c + x : before + n - 1);
      built[x] = a.chunk_state[at * per + i];
      decay[x] = a.chunk_decay[at * a.n_heads * a.D + hd];
    }
#pragma unroll
    for (int x = 0; x < CARRY_AHEAD; ++x)
      if (c + x < before + n) {
        a.chunk_state[(size_t)(c + x) * per + i] = S;
        S = fmaf(decay[x], S, built[x]);
      }
  }
  *slot = S;
}

extern "C" int llmlab_gla_slices(int D) { return (D + SLICE - 1) / SLICE; }

// proj [rows, ld] float32 holds q at off_q (heads * D), k at off_k, v at off_v (heads * E);
// decay [rows, heads * D]; state [slots, heads, D, E]; parts [rows, heads, slices, E].  kind: 0 decays per
// key channel, 1 the same with a bonus [heads * D] for the current row, 2 keep and take [rows, heads]
// in place of the decays, with the normaliser's state, pieces and (in chunks) chunk_norm.
// chunk > 0: the three-pass form over chunks of so many rows; chunk_state then holds
// max_chunks * heads * D * E floats and chunk_decay max_chunks * heads * D, with max_chunks >=
// rows / chunk + n_reqs.
extern "C" int llmlab_gla_scan(const float* proj, int ld, int off_q, int off_k, int off_v, const float* decay,
                               float q_scale, int n_heads, int D, int E, float* state, const int* q_start,
                               const int* req_rows, int n_reqs, float* parts, int rows, int chunk,
                               float* chunk_state, float* chunk_decay, int max_chunks, int kind, const float* bonus,
                               const float* keep, const float* take, float* norm_state, float* norm_parts,
                               float* chunk_norm, hipStream_t stream) {
  LLMLAB_REQUIRE(kind >= KIND_DECAY && kind <= KIND_MEMORY && (kind == KIND_MEMORY || decay) &&
                     (kind != KIND_BONUS || bonus) &&
                     (kind != KIND_MEMORY || (keep && take && norm_state && norm_parts && (chunk <= 0 || chunk_norm))),
                 "gla_scan: an operand of kind %d is missing", kind);
  LLMLAB_REQUIRE(n_reqs >= 0 && n_heads > 0 && D > 0 && E > 0, "gla_scan: bad sizes reqs=%d heads=%d D=%d E=%d", n_reqs,
                 n_heads, D, E);
  const int slices = (D + SLICE - 1) / SLICE;
  int cols = E < 64 ? E : 64;
  while (cols > 1 && slices * cols > 1024) cols /= 2;
  LLMLAB_REQUIRE(slices * cols <= 1024, "gla_scan: %d key channels per head are more than a block holds", D);
  LLMLAB_REQUIRE(n_heads <= 65535 && (E + cols - 1) / cols <= 65535 && n_reqs <= 65535,
                 "gla_scan: too many heads, columns or requests");
  if (n_reqs == 0) return 0;
  ScanArgs a{proj, ld, off_q, off_k, off_v, decay, q_scale, n_heads, D, E, cols, slices, state, q_start, req_rows, parts,
             n_reqs, chunk, chunk_state, chunk_decay, bonus, keep, take, kind == KIND_MEMORY ? norm_state : nullptr, norm_parts,
             chunk_norm};
  const bool uniform = cols == 64;
  dim3 block(slices * cols);
  const unsigned slabs = (E + cols - 1) / cols + (kind == KIND_MEMORY ? 1 : 0);
  // (blocks of up to 256 threads, heads of up to 64 key channels, are compiled with the
  // registers that leaves them: the rows fetched ahead stay in registers then)
  const bool small = slices * cols <= 256;
#define LLMLAB_SCAN_KIND(MODE, KIND, GRIDX)                                                                           \
  do {                                                                                                               \
    const dim3 grid_(GRIDX, n_heads, slabs);                                                                         \
    if (uniform && small) hipLaunchKernelGGL((gla_scan_kernel<MODE, KIND, true, 256>), grid_, block, 0, stream, a);  \
    else if (uniform) hipLaunchKernelGGL((gla_scan_kernel<MODE, KIND, true, 1024>), grid_, block, 0, stream, a);     \
    else if (small) hipLaunchKernelGGL((gla_scan_kernel<MODE, KIND, false, 256>), grid_, block, 0, stream, a);       \
    else hipLaunchKernelGGL((gla_scan_kernel<MODE, KIND, false, 1024>), grid_, block, 0, stream, a);                 \
  } while (0)
#define LLMLAB_SCAN(MODE, GRIDX)                                              \
  do {                                                                        \
    if (kind == KIND_DECAY) LLMLAB_SCAN_KIND(MODE, KIND_DECAY, GRIDX);        \
    else if (kind == KIND_BONUS) LLMLAB_SCAN_KIND(MODE, KIND_BONUS, GRIDX);   \
    else LLMLAB_SCAN_KIND(MODE, KIND_MEMORY, GRIDX);                          \
  } while (0)
  if (chunk <= 0) {
    LLMLAB_SCAN(SCAN_WHOLE, n_reqs);
  } else {
    const int chunks = rows / chunk + n_reqs;
    LLMLAB_REQUIRE(chunk_state && chunk_decay && max_chunks >= chunks,
                   "gla_scan: %d rows of %d requests in chunks of %d need room for %d chunks, got %d", rows, n_reqs,
                   chunk, chunks, max_chunks);
    LLMLAB_SCAN(SCAN_LOCAL, chunks);
    const size_t per = (size_t)n_heads * D * E + (kind == KIND_MEMORY ? (size_t)n_heads * D : 0);
    hipLaunchKernelGGL(gla_carry_kernel, dim3((unsigned)((per + 255) / 256), n_reqs), dim3(256), 0, stream, a);
    LLMLAB_SCAN(SCAN_FINISH, chunks);
  }
#undef LLMLAB_SCAN
#undef LLMLAB_SCAN_KIND
  LLMLAB_LAUNCH_CHECK("gla_scan");
  return 0;
}

// ---------------------------------------------------------------------- output
// Block (row, head): o = sum over slices of parts; y = o / sqrt(mean(o^2) + eps) * w[e]
// (the weight has one entry per value channel, the same for every head; w_per_head: one per
// head and channel, w[h * E + e]); out = T(y * silu(gate)), silu(g) = g / (1 + exp(-g))
// (gate_kind 1: y * sigmoid(gate)); gate [rows, ld] float32 at column off_g.  norm_parts [rows, heads,
// slices] and maxima [rows, heads] (a memory with a normaliser): o is first divided by max(|n . q|,
// exp(-m)) + 1e-6, n . q the sum of its parts.
__device__ __forceinline__ float memory_size(float nq, float m) { return fmaxf(fabsf(nq), expf(-m)) + 1e-6f; }
template <typename T>
__global__ __launch_bounds__(1024) void gla_output_kernel(const float* __restrict__ parts, int slices, int n_heads, int E,
                                                          const float* __restrict__ w, float eps,
                                                          const float* __restrict__ proj, int ld, int off_g,
                                                          T* __restrict__ out, int w_per_head, int gate_kind,
                                                          int count, const float* __restrict__ norm_parts,
                                                          const float* __restrict__ maxima) {
  __shared__ float red[17];
  const int r = blockIdx.x, h = blockIdx.y, e = threadIdx.x;
  float o = 0.f;
  if (e < E) {
    const float* p = parts + (((size_t)r * n_heads + h) * slices) * E + e;
    for (int s = 0; s < slices; ++s) o += p[(size_t)s * E];
  }
  if (norm_parts) {
    const float* n = norm_parts + ((size_t)r * n_heads + h) * slices;
    float nq = 0.f;
    for (int s = 0; s < slices; ++s) nq += n[s];
    o = o / memory_size(nq, maxima[(size_t)r * n_heads + h]);
  }
  const float ms = block_sum(o * o, red) / (float)count;      // (count < E: the channels behind it are zeros)
  if (e < E) {
    const float g = proj[(size_t)r * ld + off_g + h * E + e];
    const float y = o * (1.0f / sqrtf(ms + eps)) * w[w_per_head ? h * E + e : e];
    const float sg = 1.0f / (1.0f + expf(-g));
    out[((size_t)r * n_heads + h) * E + e] = from_float<T>(y * (gate_kind == 1 ? sg : g * sg));
  }
}

// slices > 0: that many pieces per output (0: as the gated scan leaves them, one per SLICE key channels);
// norm_count > 0: the mean of the squares is taken over so many channels (the others are zeros)
extern "C" int llmlab_gla_output(const float* parts, int rows, int n_heads, int D, int E, const float* w, float eps,
                                 const float* proj, int ld, int off_g, void* out, int dtype, int slices_given,
                                 int w_per_head, int gate_kind, int norm_count, const float* norm_parts,
                                 const float* maxima, hipStream_t stream) {
  LLMLAB_REQUIRE((norm_parts == nullptr) == (maxima == nullptr), "gla_output: a normaliser comes with its maxima");
  LLMLAB_REQUIRE(rows >= 0 && n_heads > 0 && n_heads <= 65535 && E > 0 && E <= 1024,
                 "gla_output: bad sizes rows=%d heads=%d E=%d", rows, n_heads, E);
  LLMLAB_REQUIRE(gate_kind == 0 || gate_kind == 1, "gla_output: unknown gate %d", gate_kind);
  LLMLAB_REQUIRE(norm_count >= 0 && norm_count <= E, "gla_output: a mean over %d of %d channels", norm_count, E);
  const int count = norm_count > 0 ? norm_count : E;
  if (rows == 0) return 0;
  const int slices = slices_given > 0 ? slices_given : (D + SLICE - 1) / SLICE;
  dim3 grid(rows, n_heads), block((E + 63) / 64 * 64);
  if (dtype == DT_BF16)
    hipLaunchKernelGGL(gla_output_kernel<bf16_t>, grid, block, 0, stream, parts, slices, n_heads, E, w, eps, proj, ld,
                       off_g, (bf16_t*)out, w_per_head, gate_kind, count, norm_parts, maxima);
  else
    hipLaunchKernelGGL(gla_output_kernel<float>, grid, block, 0, stream, parts, slices, n_heads, E, w, eps, proj, ld,
                       off_g, (float*)out, w_per_head, gate_kind, count, norm_parts, maxima);
  LLMLAB_LAUNCH_CHECK("gla_output");
  return 0;
}


// ------------------------------------------------------------------ chunks on the matrix cores
// Long portions, all three kinds, as products of 64-row chunks (float32 matrix instructions,
// v_mfma_f32_16x16x4_f32: 32-bit products and sums), in the same three passes as above:
//   LOCAL   per chunk and head: L = sum_s diag(decays behind s) k_s v_s^T as one product [D x 64] [64 x E];
//   carry   (gla_carry_kernel);
//   FINISH  per chunk and head, a wave 16 rows t: o_t = (decayed q_t)^T S_start + sum_(s <= t) p_ts v_s with the
//           pair weights p_ts = sum_d q_t[d] k_s[d] (product of the decays a_u[d], s < u <= t), then the head's
//           norm, its gate and the rounding (the output kernel's work) while the outputs are in registers.
// Products of decays are taken as 2^(difference of sums of logarithms).  A sum covers at most the 16
// rows of a sub-block; across sub-blocks the sub-blocks' totals are added, so that the terms of a
// difference stay small and every exponent is at most 0: nothing overflows, and the ratio of two
// neighbours is exact to a few units of a sum over 16 rows.  Pairs in different sub-blocks: their
// decays split at the later sub-block's start into a factor of k_s and a factor of q_t, and the weights
// are a matrix product.  Pairs in one sub-block: a lane takes the row t = lane % 16 and four rows s and
// walks the key channels.  MEMORY has one decay per head: all its weights are products q_t . k_s times a
// number per pair, and the normaliser's n_t . q_t is their sum.
// The weights are taken transposed (rows s, columns t): an accumulator then is the next product's operand,
// lane (t, g) holding s = 4 g + r in register r.
struct ChunkArgs {
  const float* proj; int ld, off_q, off_k, off_v, off_g; float q_scale; int n_heads, D, E;
  const float* logs;                              // log2 of the decays: [rows, heads, D], or (MEMORY) [rows, heads]
  const float* take; const float* bonus;          // MEMORY: [rows, heads]; BONUS: [heads, D]
  const int* q_start; int n_reqs;
  float* chunk_state; float* chunk_decay; float* chunk_norm;
  const float* w; float eps; int w_per_head, gate_kind, count; const float* maxima;
};
constexpr int CK = 64, SUB = 16;
__device__ __forceinline__ float exp2_(float x) { return __builtin_amdgcn_exp2f(x); }

__device__ __forceinline__ bool chunk_rows(const int* __restrict__ q_start, int n_reqs, int index, int& first, int& n) {
  int before = 0;
  for (int b = 0; b < n_reqs; ++b) {
    const int lo = q_start[b], hi = q_start[b + 1], chunks = (hi - lo + CK - 1) / CK;
    if (index < before + chunks) {
      first = lo + (index - before) * CK;
      n = hi - first < CK ? hi - first : CK;
      return true;
    }
    before += chunks;
  }
  return false;
}

// The sums of the logs within each sub-block (inclusive) to s_lb[row * stride + d], the sub-blocks' totals to
// s_tot[sub * width + d]; channels d < width (width 1: MEMORY's one number a row, log_ld numbers apart).
// Rows past the chunk's end do not decay; channels from D to width are zeros.
__device__ __forceinline__ void chunk_log_sums(const float* __restrict__ logs, size_t log_ld, int D, int width, int n,
                                               float* s_lb, int stride, float* s_tot) {
  for (int c = threadIdx.x; c < (CK / SUB) * width; c += blockDim.x) {
    const int sub = c / width, d = c - sub * width;
    float lg[SUB], sum = 0.f;
#pragma unroll
    for (int i = 0; i < SUB; ++i) {              // (past the end: the last ones, set aside below; no load under a branch)
      const int row = sub * SUB + i;
      lg[i] = logs[(size_t)(row < n ? row : n - 1) * log_ld + (d < D ? d : D - 1)];
    }
#pragma unroll
    for (int i = 0; i < SUB; ++i) {
      sum += (sub * SUB + i < n && d < D) ? lg[i] : 0.f;
      s_lb[(sub * SUB + i) * stride + d] = sum;
    }
    s_tot[sub * width + d] = sum;
  }
}

// Operands of the products lie in LDS in rows of a multiple of 64 floats plus 16: the lanes (c, g) of a read
// then are 16 consecutive numbers of four rows in all 64 banks.  Values and states pass through one buffer
// SLAB columns at a time; a slab's numbers are asked for into registers while the products before it run.
constexpr int SLAB = 64, SLAB_STRIDE = SLAB + 16;
__host__ __device__ inline int product_stride(int columns) { return (columns + 63) / 64 * 64 + 16; }
// the slab e0 .. of the chunk's values (this thread's 16 numbers: one row of 64 columns a wave at a time)
__device__ __forceinline__ void fetch_values(const ChunkArgs& a, int first, int n, int h, int e0, float (&reg)[16]) {
  const int e = e0 + (int)(threadIdx.x & 63), ec = e < a.E ? e : a.E - 1;
#pragma unroll
  for (int i = 0; i < 16; ++i) {
    const int s = 4 * i + (int)(threadIdx.x >> 6);      // (past the end: the last row, which weighs nothing)
    reg[i] = a.proj[(size_t)(first + (s < n ? s : n - 1)) * a.ld + a.off_v + h * a.E + ec];
  }
}
__device__ __forceinline__ void stash_slab(float* buf, const float (&reg)[16], int row0) {
#pragma unroll
  for (int i = 0; i < 16; ++i) buf[(row0 + 4 * i + (int)(threadIdx.x >> 6)) * SLAB_STRIDE + (int)(threadIdx.x & 63)] = reg[i];
}

template <int KIND>
__global__ __launch_bounds__(256) void chunk_local_kernel(ChunkArgs a) {
  extern __shared__ __attribute__((aligned(16))) float chunk_lds[];
  int first, n;
  if (!chunk_rows(a.q_start, a.n_reqs, blockIdx.x, first, n)) return;
  const int h = blockIdx.y, D = a.D, E = a.E, DK = (D + 15) & ~15, KS = product_stride(DK);
  const int width = KIND == KIND_MEMORY ? 1 : DK;
  float* s_k = chunk_lds;                        // the decayed keys [64][KS]
  float* s_v = s_k + CK * KS;                    // a slab of the values [64][SLAB_STRIDE]
  float* s_tot = s_v + CK * SLAB_STRIDE;         // totals of the sub-blocks' logs [4][width]
  float* s_lb = s_tot + 4 * width;               // MEMORY: the sums of the logs and takes [64] [64]
  float vreg[16];
  fetch_values(a, first, n, h, 0, vreg);
  constexpr int ITEMS = 2;                       // (sub-block, key channel) pairs a thread takes: D <= 128
  float lb[KIND == KIND_MEMORY ? 1 : ITEMS][SUB], kk[ITEMS][SUB];
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
    const int item = threadIdx.x + 256 * it, sub = item / DK, d = item - sub * DK;
    if (sub < 4) {
      const int dc = d < D ? d : D - 1;
#pragma unroll
      for (int i = 0; i < SUB; ++i) {            // (rows past the end: the last one, set aside below)
        const int row = sub * SUB + i, rc = first + (row < n ? row : n - 1);
        kk[it][i] = a.proj[(size_t)rc * a.ld + a.off_k + h * D + dc];
        if (KIND != KIND_MEMORY) lb[it][i] = a.logs[((size_t)rc * a.n_heads + h) * D + dc];
      }
      if (KIND != KIND_MEMORY) {
        float sum = 0.f;
#pragma unroll
        for (int i = 0; i < SUB; ++i) {
          sum += (sub * SUB + i < n && d < D) ? lb[it][i] : 0.f;
          lb[it][i] = sum;
        }
        s_tot[sub * width + d] = sum;
      }
    }
  }
  if (KIND == KIND_MEMORY) {
    chunk_log_sums(a.logs + (size_t)first * a.n_heads + h, a.n_heads, 1, 1, n, s_lb, 1, s_tot);
    if (threadIdx.x < CK) s_lb[CK + threadIdx.x] = (int)threadIdx.x < n ? a.take[(size_t)(first + threadIdx.x) * a.n_heads + h] : 0.f;
  }
  __syncthreads();
  const size_t at = (size_t)blockIdx.x * a.n_heads + h;
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
    const int item = threadIdx.x + 256 * it, sub = item / DK, d = item - sub * DK;
    if (sub < 4) {
      const int dl = KIND == KIND_MEMORY ? 0 : d;
      float tail = s_tot[sub * width + dl];      // from the sub-block's start to the chunk's end
      for (int b = sub + 1; b < 4; ++b) tail += s_tot[b * width + dl];
#pragma unroll
      for (int i = 0; i < SUB; ++i) {
        const int row = sub * SUB + i;
        float k = (row < n && d < D) ? kk[it][i] : 0.f;
        if (KIND == KIND_MEMORY) k *= exp2_(tail - s_lb[row]) * s_lb[CK + row];
        else k *= exp2_(tail - lb[it][i]);
        s_k[row * KS + d] = k;
      }
      if (sub == 0 && d < D) a.chunk_decay[at * D + d] = exp2_(tail);
    }
  }
  stash_slab(s_v, vreg, 0);
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c = lane & 15, g = lane >> 4;
  const int tiles = DK / 16, steps = (n + 15) >> 4 << 2;      // (four rows a step, steps in fours)
  float* out = a.chunk_state + at * D * E;
  for (int e0 = 0; e0 < E; e0 += SLAB) {
    const bool more = e0 + SLAB < E;
    if (more) fetch_values(a, first, n, h, e0 + SLAB, vreg);
    for (int item = wave; item < 2 * tiles; item += 4) {      // a tile of 16 key channels x half the slab
      const int dt = item >> 1, half = (item & 1) * 32;
      if (e0 + half >= E) continue;
      floatx4 acc[2] = {floatx4{0.f, 0.f, 0.f, 0.f}, floatx4{0.f, 0.f, 0.f, 0.f}};
      for (int q0 = 0; q0 < steps; q0 += 4)
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int q = q0 + u;
        const float k = s_k[(4 * q + g) * KS + dt * 16 + c];
        const float* v = s_v + (4 * q + g) * SLAB_STRIDE + half + c;
        acc[0] = __builtin_amdgcn_mfma_f32_16x16x4f32(k, v[0], acc[0], 0, 0, 0);
        acc[1] = __builtin_amdgcn_mfma_f32_16x16x4f32(k, v[16], acc[1], 0, 0, 0);
      }
#pragma unroll
      for (int x = 0; x < 2; ++x)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int row = dt * 16 + 4 * g + r, e = e0 + half + 16 * x + c;
          if (row < D && e < E) out[(size_t)row * E + e] = acc[x][r];
        }
    }
    __syncthreads();
    if (!more) break;
    stash_slab(s_v, vreg, 0);
    __syncthreads();
  }
  if (KIND == KIND_MEMORY)
    for (int d = threadIdx.x; d < D; d += 256) {
      float sum = 0.f;
      for (int s = 0; s < n; ++s) sum += s_k[s * KS + d];
      a.chunk_norm[at * D + d] = sum;
    }
}

template <int KIND, int ET, typename T>
__global__ __launch_bounds__(256) void chunk_finish_kernel(ChunkArgs a, T* __restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) float chunk_lds[];
  int first, n;
  if (!chunk_rows(a.q_start, a.n_reqs, blockIdx.x, first, n)) return;
  const int h = blockIdx.y, D = a.D, E = a.E, DK = (D + 15) & ~15, DS = DK + 4;
  const int width = KIND == KIND_MEMORY ? 1 : DK, stride = KIND == KIND_MEMORY ? 1 : DS;
  float* s_q = chunk_lds;
  float* s_k = s_q + CK * DS;
  float* s_lb = s_k + CK * DS;
  float* s_tot = s_lb + CK * stride;
  float* s_one = s_tot + 4 * (width > 4 ? width : 4);      // BONUS: the bonus [DK]; MEMORY: the normaliser [DK], takes [64]
  float* s_buf = s_one + DK + CK;                            // a slab of the state [DK] or of the values [64]
  const size_t at = (size_t)blockIdx.x * a.n_heads + h;
  const float* S0 = a.chunk_state + at * D * E;
  // a slab of the state: 64 rows d a time, as many times as it takes
  auto fetch_state = [&](int d0, int e0, float (&reg)[16]) {
    const int e = e0 + (int)(threadIdx.x & 63), ec = e < E ? e : E - 1;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int d = d0 + 4 * i + (int)(threadIdx.x >> 6);      // (past the end: the last row, which meets zeros)
      reg[i] = S0[(size_t)(d < D ? d : D - 1) * E + ec];
    }
  };
  float sreg[2][16], vreg[16];
  fetch_state(0, 0, sreg[0]);
  if (DK > 64) fetch_state(64, 0, sreg[1]);
  for (int i0 = 0; i0 < CK * DK; i0 += 1024)
#pragma unroll
  for (int u = 0; u < 4; ++u) {                  // (CK * DK is a multiple of 1,024)
    const int i = i0 + 256 * u + (int)threadIdx.x;
    const int row = i / DK, d = i - row * DK;
    const bool in = row < n && d < D;
    const float* p = a.proj + (size_t)(first + (row < n ? row : n - 1)) * a.ld + h * D + (d < D ? d : D - 1);
    const float q = p[a.off_q], k = p[a.off_k];
    s_q[row * DS + d] = in ? q * a.q_scale : 0.f;
    s_k[row * DS + d] = in ? k : 0.f;
  }
  if (KIND == KIND_MEMORY) chunk_log_sums(a.logs + (size_t)first * a.n_heads + h, a.n_heads, 1, 1, n, s_lb, 1, s_tot);
  else chunk_log_sums(a.logs + ((size_t)first * a.n_heads + h) * D, (size_t)a.n_heads * D, D, DK, n, s_lb, stride, s_tot);
  if (KIND != KIND_DECAY)
    for (int d = threadIdx.x; d < DK; d += 256) {
      const int dc = d < D ? d : D - 1;
      s_one[d] = d < D ? (KIND == KIND_BONUS ? a.bonus[h * D + dc] : a.chunk_norm[at * D + dc]) : 0.f;
    }
  if (KIND == KIND_MEMORY && threadIdx.x < CK) {
    const int row = (int)threadIdx.x;
    s_one[DK + row] = row < n ? a.take[(size_t)(first + row) * a.n_heads + h] : 0.f;
  }
  auto stash_state = [&]() {
    stash_slab(s_buf, sreg[0], 0);
    if (DK > 64) stash_slab(s_buf, sreg[1], 64);
  };
  stash_state();
  __syncthreads();
  fetch_values(a, first, n, h, 0, vreg);
  const int lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
  const int i0 = __builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6));      // this wave's sub-block
  const bool busy = i0 * SUB < n;                // (a wave without rows takes part in the barriers only)
  const int t = i0 * SUB + c;                    // this lane's row (as a row of an operand)
  const float* q_t = s_q + t * DS;
  // the sum of the logs from the sub-block's start that row t's outputs see (BONUS: up to the row before)
  auto seen = [&](int d) {
    if (KIND == KIND_BONUS) return c == 0 ? 0.f : s_lb[(t - 1) * stride + d];
    return s_lb[t * stride + (KIND == KIND_MEMORY ? 0 : d)];
  };
  // ---- the weights of row t and the rows s = 16 j + 4 g + r of the chunk
  floatx4 p[4];
  float nq = 0.f;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    p[j] = floatx4{0.f, 0.f, 0.f, 0.f};
    if (!busy || j > i0) continue;
    if (KIND == KIND_MEMORY) {
      for (int k0 = 0; k0 < DK; k0 += 16)
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          const int d = k0 + 4 * u + g;
          p[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(s_k[(j * SUB + c) * DS + d], q_t[d], p[j], 0, 0, 0);
        }
      float between = 0.f;                       // from the end of s's sub-block on (or, in one sub-block, nothing)
      for (int b = j + 1; b < i0; ++b) between += s_tot[b];
      const float base = seen(0) + between + (j < i0 ? s_tot[j] : 0.f);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int s = j * SUB + 4 * g + r;
        p[j][r] = s <= t ? p[j][r] * exp2_(fminf(base - s_lb[s], 0.f)) * s_one[DK + s] : 0.f;
        nq += p[j][r];
      }
    } else if (j < i0) {
      for (int k0 = 0; k0 < DK; k0 += 16)
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int d = k0 + 4 * u + g;
        float lg = s_tot[j * width + d] - s_lb[(j * SUB + c) * stride + d];
        for (int b = j + 1; b < i0; ++b) lg += s_tot[b * width + d];
        p[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(s_k[(j * SUB + c) * DS + d] * exp2_(lg), q_t[d] * exp2_(seen(d)), p[j], 0, 0, 0);
      }
    } else {
      const int s0 = j * SUB + 4 * g;
      for (int d = 0; d < DK; d += 4) {
        const floatx4 q4 = *(const floatx4*)(q_t + d);
        floatx4 see4;
        if (KIND == KIND_BONUS && c == 0) see4 = floatx4{0.f, 0.f, 0.f, 0.f};
        else see4 = *(const floatx4*)(s_lb + (KIND == KIND_BONUS ? t - 1 : t) * stride + d);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const floatx4 k4 = *(const floatx4*)(s_k + (s0 + r) * DS + d);
          const floatx4 lb4 = *(const floatx4*)(s_lb + (s0 + r) * stride + d);
#pragma unroll
          for (int x = 0; x < 4; ++x) p[j][r] = fmaf(q4[x] * k4[x], exp2_(fminf(see4[x] - lb4[x], 0.f)), p[j][r]);
        }
      }
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (s0 + r > t || (KIND == KIND_BONUS && s0 + r == t)) p[j][r] = 0.f;
      if (KIND == KIND_BONUS) {                  // the row itself, through the bonus: a quarter of the channels a lane
        float own = 0.f;
        for (int d = g; d < DK; d += 4) own = fmaf(q_t[d] * s_k[t * DS + d], s_one[d], own);
        own += __shfl_xor(own, 16, WAVE);
        own += __shfl_xor(own, 32, WAVE);
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (s0 + r == t) p[j][r] = own;
      }
    }
  }
  // ---- slab by slab: what the state before the chunk gives, and what the chunk's rows give
  floatx4 acc[ET];
#pragma unroll
  for (int et = 0; et < ET; ++et) acc[et] = floatx4{0.f, 0.f, 0.f, 0.f};
  auto slab = [&](auto number) {                 // (returns whether there is another one behind it)
    constexpr int TILES = ET < 4 ? ET : 4, X0 = 4 * decltype(number)::value, e0 = 16 * X0;
    const bool more = X0 + 4 < ET && e0 + SLAB < E;
    if (busy) {
      for (int k0 = 0; k0 < DK; k0 += 16)
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int d = k0 + 4 * u + g, dl = KIND == KIND_MEMORY ? 0 : d;
        float lg = seen(d);
        for (int j = 0; j < i0; ++j) lg += s_tot[j * width + dl];
        const float q = q_t[d] * exp2_(lg);
        if (KIND == KIND_MEMORY && e0 == 0) nq = fmaf(q, s_one[d], nq);
        const float* srow = s_buf + d * SLAB_STRIDE + c;
#pragma unroll
        for (int x = 0; x < TILES; ++x)
          acc[X0 + x] = __builtin_amdgcn_mfma_f32_16x16x4f32(q, srow[16 * x], acc[X0 + x], 0, 0, 0);
      }
    }
    __syncthreads();
    stash_slab(s_buf, vreg, 0);
    __syncthreads();
    if (more) {
      fetch_state(0, e0 + SLAB, sreg[0]);
      if (DK > 64) fetch_state(64, e0 + SLAB, sreg[1]);
    }
    if (busy) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        if (j > i0) continue;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float* v = s_buf + (j * SUB + 4 * g + r) * SLAB_STRIDE + c;
#pragma unroll
          for (int x = 0; x < TILES; ++x)
            acc[X0 + x] = __builtin_amdgcn_mfma_f32_16x16x4f32(p[j][r], v[16 * x], acc[X0 + x], 0, 0, 0);
        }
      }
    }
    if (!more) return false;
    __syncthreads();
    stash_state();
    __syncthreads();
    fetch_values(a, first, n, h, e0 + SLAB, vreg);
    return true;
  };
  bool again = slab(std::integral_constant<int, 0>{});
  if constexpr (ET > 4) again = again && slab(std::integral_constant<int, 1>{});
  if constexpr (ET > 8) again = again && slab(std::integral_constant<int, 2>{});
  if constexpr (ET > 12) again = again && slab(std::integral_constant<int, 3>{});
  if (!busy) return;
  // ---- norm, gate, rounding: this lane now holds the columns 16 et + c of the rows 4 g + r
  // (all gates and weights are asked for together; past the end the last ones, dropped)
  float gates[ET][4], ws[ET];
#pragma unroll
  for (int et = 0; et < ET; ++et) {
    const int e = 16 * et + c < E ? 16 * et + c : E - 1;
    ws[et] = a.w[a.w_per_head ? h * E + e : e];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = i0 * SUB + 4 * g + r;
      gates[et][r] = a.proj[(size_t)(first + (row < n ? row : n - 1)) * a.ld + a.off_g + h * E + e];
    }
  }
  if (KIND == KIND_MEMORY) {
    nq += __shfl_xor(nq, 16, WAVE);
    nq += __shfl_xor(nq, 32, WAVE);
  }
  float inv[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int row = i0 * SUB + 4 * g + r;
    if (KIND == KIND_MEMORY) {
      const float size = memory_size(__shfl(nq, 4 * g + r, WAVE), a.maxima[(size_t)(first + (row < n ? row : n - 1)) * a.n_heads + h]);
#pragma unroll
      for (int et = 0; et < ET; ++et) acc[et][r] /= size;
    }
    float ss = 0.f;
#pragma unroll
    for (int et = 0; et < ET; ++et) ss = fmaf(acc[et][r], 16 * et + c < E ? acc[et][r] : 0.f, ss);
#pragma unroll
    for (int off = 8; off > 0; off >>= 1) ss += __shfl_xor(ss, off, WAVE);
    inv[r] = 1.0f / sqrtf(ss / (float)a.count + a.eps);
  }
#pragma unroll
  for (int et = 0; et < ET; ++et) {
    const int e = 16 * et + c;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = i0 * SUB + 4 * g + r;
      const float gate = gates[et][r];
      const float sg = 1.0f / (1.0f + expf(-gate));
      const T y = from_float<T>(acc[et][r] * inv[r] * ws[et] * (a.gate_kind == 1 ? sg : gate * sg));
      if (row < n && e < E) out[((size_t)(first + row) * a.n_heads + h) * E + e] = y;
    }
  }
}

constexpr int CHUNK_MAX_D = 128, CHUNK_MAX_E = 256, CHUNK_MAX_LDS = 152 * 1024;
extern "C" int llmlab_chunk_scan_takes(int D, int E) { return D > 0 && E > 0 && D <= CHUNK_MAX_D && E <= CHUNK_MAX_E; }
extern "C" int llmlab_chunk_scan_rows() { return CK; }

// From the projections and the logarithms of the decays to the gated outputs (as gla_scan and gla_output).
// chunk_state [max_chunks, heads, D, E], chunk_decay and (memory) chunk_norm [max_chunks, heads, D], with
// max_chunks >= rows / CK + n_reqs.
extern "C" int llmlab_chunk_scan(const float* proj, int ld, int off_q, int off_k, int off_v, int off_g, float q_scale,
                                 int n_heads, int D, int E, const float* logs, float* state, const int* q_start,
                                 const int* req_rows, int n_reqs, int rows, int kind, const float* bonus, const float* take,
                                 float* norm_state, const float* maxima, float* chunk_state, float* chunk_decay,
                                 float* chunk_norm, int max_chunks, const float* w, float eps, int w_per_head, int gate_kind,
                                 int norm_count, void* out, int dtype, hipStream_t stream) {
  LLMLAB_REQUIRE(llmlab_chunk_scan_takes(D, E) && n_heads > 0 && n_heads <= 65535 && n_reqs >= 0 && n_reqs <= 65535 && rows >= 0,
                 "chunk_scan: sizes D=%d E=%d heads=%d are not taken", D, E, n_heads);
  LLMLAB_REQUIRE(ld >= off_q + n_heads * D && ld >= off_k + n_heads * D && ld >= off_v + n_heads * E &&
                     ld >= off_g + n_heads * E && off_q >= 0 && off_k >= 0 && off_v >= 0 && off_g >= 0,
                 "chunk_scan: rows of %d numbers do not hold the projections", ld);
  LLMLAB_REQUIRE(proj && logs && state && q_start && req_rows && chunk_state && chunk_decay && w && out &&
                     norm_count >= 0 && norm_count <= E && (gate_kind == 0 || gate_kind == 1) &&
                     kind >= KIND_DECAY && kind <= KIND_MEMORY && (kind != KIND_BONUS || bonus) &&
                     (kind != KIND_MEMORY || (take && norm_state && maxima && chunk_norm)),
                 "chunk_scan: an operand of kind %d is missing", kind);
  if (rows == 0 || n_reqs == 0) return 0;
  const int chunks = rows / CK + n_reqs;
  LLMLAB_REQUIRE(max_chunks >= chunks, "chunk_scan: %d rows of %d requests need room for %d chunks, got %d", rows, n_reqs,
                 chunks, max_chunks);
  const ChunkArgs a{proj, ld, off_q, off_k, off_v, off_g, q_scale, n_heads, D, E, logs, take, bonus, q_start, n_reqs,
                    chunk_state, chunk_decay, chunk_norm, w, eps, w_per_head, gate_kind, norm_count > 0 ? norm_count : E,
                    maxima};
  const int DK = (D + 15) & ~15, et = (E + 15) / 16;
  const size_t lds_local = ((size_t)CK * product_stride(DK) + (size_t)CK * SLAB_STRIDE + 4 * DK + 2 * CK) * sizeof(float);
  const size_t lds_finish = ((size_t)(kind == KIND_MEMORY ? 2 : 3) * CK * (DK + 4) + CK + 4 * DK + 16 +
                             DK + (DK > CK ? 2 * CK : CK) * SLAB_STRIDE) * sizeof(float);
  const dim3 grid(chunks, n_heads), block(256);
  // (LDS beyond 64 KB is asked for once per kernel)
#define LLMLAB_CHUNK_LDS(KERNEL, BYTES)                                                                                   \
  do {                                                                                                                    \
    static bool raised = false;                                                                                           \
    if ((BYTES) > 64 * 1024 && !raised) {                                                                                 \
      LLMLAB_REQUIRE(hipFuncSetAttribute((const void*)KERNEL, hipFuncAttributeMaxDynamicSharedMemorySize,                 \
                                         CHUNK_MAX_LDS) == hipSuccess, "chunk_scan: no %zu bytes of LDS", (size_t)(BYTES)); \
      raised = true;                                                                                                      \
    }                                                                                                                     \
  } while (0)
#define LLMLAB_CHUNK_FINISH(KIND, ETV, T)                                                                                 \
  do {                                                                                                                    \
    auto kernel = chunk_finish_kernel<KIND, ETV, T>;                                                                      \
    LLMLAB_CHUNK_LDS(kernel, lds_finish);                                                                                 \
    hipLaunchKernelGGL(kernel, grid, block, lds_finish, stream, a, (T*)out);                                              \
  } while (0)
#define LLMLAB_CHUNK_LOCAL(KIND)                                              \
  do {                                                                        \
    auto kernel = chunk_local_kernel<KIND>;                                   \
    LLMLAB_CHUNK_LDS(kernel, lds_local);                                      \
    hipLaunchKernelGGL(kernel, grid, block, lds_local, stream, a);            \
  } while (0)
#define LLMLAB_CHUNK(KIND, ETV)                                                                                  \
  do {                                                                                                           \
    if (dtype == DT_BF16) LLMLAB_CHUNK_FINISH(KIND, ETV, bf16_t);                                           \
    else LLMLAB_CHUNK_FINISH(KIND, ETV, float);                                                                  \
  } while (0)
#define LLMLAB_CHUNK_ET(KIND)                 \
  do {                                        \
    if (et <= 2) LLMLAB_CHUNK(KIND, 2);       \
    else if (et <= 4) LLMLAB_CHUNK(KIND, 4);  \
    else if (et <= 8) LLMLAB_CHUNK(KIND, 8);  \
    else LLMLAB_CHUNK(KIND, 16);              \
  } while (0)
  if (kind == KIND_DECAY) LLMLAB_CHUNK_LOCAL(KIND_DECAY);
  else if (kind == KIND_BONUS) LLMLAB_CHUNK_LOCAL(KIND_BONUS);
  else LLMLAB_CHUNK_LOCAL(KIND_MEMORY);
  ScanArgs carry{};
  carry.n_heads = n_heads; carry.D = D; carry.E = E; carry.state = state; carry.q_start = q_start; carry.req_rows = req_rows;
  carry.n_reqs = n_reqs; carry.chunk = CK; carry.chunk_state = chunk_state; carry.chunk_decay = chunk_decay;
  carry.norm_state = kind == KIND_MEMORY ? norm_state : nullptr; carry.chunk_norm = chunk_norm;
  const size_t per = (size_t)n_heads * D * E + (kind == KIND_MEMORY ? (size_t)n_heads * D : 0);
  hipLaunchKernelGGL(gla_carry_kernel, dim3((unsigned)((per + 255) / 256), n_reqs), dim3(256), 0, stream, carry);
  if (kind == KIND_DECAY) LLMLAB_CHUNK_ET(KIND_DECAY);
  else if (kind == KIND_BONUS) LLMLAB_CHUNK_ET(KIND_BONUS);
  else LLMLAB_CHUNK_ET(KIND_MEMORY);
#undef LLMLAB_CHUNK_ET
#undef LLMLAB_CHUNK
#undef LLMLAB_CHUNK_LOCAL
#undef LLMLAB_CHUNK_FINISH
#undef LLMLAB_CHUNK_LDS
  LLMLAB_LAUNCH_CHECK("chunk_scan");
  return 0;
}

// ------------------------------------------------------------------ one row, whole
// Decoding: every request brings ONE row.  A block takes a request's row for one head and does what
// the decays (or gates), the scan and the output do in three launches: the state [D, E] comes from the
// slot into registers (a group of E / 4 lanes a key channel, four value channels a lane, the loads
// asked for before anything else), meanwhile the decays of the head's key channels (or its gates) are worked
// out, then the update, the read-out, the sum over the groups through LDS, the head's norm and its gate.
// The same numbers as the three kernels up to the order of the sums over key channels.
struct RowArgs {
  const float* proj; int ld, off_q, off_k, off_v, off_g; float q_scale; int n_heads, D, E, groups;
  float* state; const int* q_start; const int* req_rows;
  const float* w; float eps; int w_per_head, gate_kind, count;
  int off_low, rank; const float* w2; const float* bias; int decay_kind; float inv_tau;      // DECAY, BONUS
  const float* bonus;                                                                         // BONUS
  int off_i, off_f; const float* bias_i; const float* bias_f; float cap; float* norm_state; float* max_state;      // MEMORY
};
constexpr int ROW_MAX_RANK = 512;
template <int KIND, typename T, int ROWS>      // ROWS: key channels a group of lanes takes at most
__global__ __launch_bounds__(1024) void recurrent_row_kernel(RowArgs a, T* __restrict__ out) {
  extern __shared__ float row_lds[];           // low [rank] | q, k, decay, bonus [D each] | sums [groups, E]
  __shared__ float red[17];
  const int b = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, D = a.D, E = a.E;
  const int r = a.q_start[b], slot = a.req_rows[b];
  const float* row = a.proj + (size_t)r * a.ld;
  float* s_low = row_lds;
  float* s_q = row_lds + (KIND == KIND_MEMORY ? 0 : a.rank);
  float* s_k = s_q + D;
  float* s_a = s_k + D;
  float* s_u = s_a + D;
  float* s_sum = s_u + D;
  const int lanes = E >> 2, g = tid / lanes, j = tid - g * lanes;
  const bool active = g < a.groups;
  float* st = a.state + ((size_t)slot * a.n_heads + h) * D * E + 4 * j;
  floatx4 S[ROWS];
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {             // (past the end: the last channel again, dropped below)
    const int d = min(g + a.groups * i, D - 1);
    S[i] = active ? *(const floatx4*)(st + (size_t)d * E) : floatx4{0.f, 0.f, 0.f, 0.f};
  }
  floatx4 v = floatx4{0.f, 0.f, 0.f, 0.f};
  if (active)
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = row[a.off_v + h * E + 4 * j + i];
  const float gate = tid < E ? row[a.off_g + h * E + tid] : 0.f;
  const float w = tid < E ? a.w[a.w_per_head ? h * E + tid : tid] : 0.f;
  for (int d = tid; d < D; d += blockDim.x) {
    s_q[d] = row[a.off_q + h * D + d];
    s_k[d] = row[a.off_k + h * D + d];
    if (KIND == KIND_BONUS) s_u[d] = a.bonus[h * D + d];
  }
  float keep = 0.f, m = 0.f;
  if (KIND == KIND_MEMORY) {                   // (a head's two gates: every thread for itself)
    const float before = a.max_state[(size_t)slot * a.n_heads + h];
    const float in = a.cap * tanhf((row[a.off_i + h] + (a.bias_i ? a.bias_i[h] : 0.f)) / a.cap);
    const float z = a.cap * tanhf((row[a.off_f + h] + (a.bias_f ? a.bias_f[h] : 0.f)) / a.cap);
    const float f = -(fmaxf(-z, 0.f) + log1pf(expf(-fabsf(z))));
    m = fmaxf(f + before, in);
    keep = expf(f + before - m);
    const float take = expf(in - m);
    v *= take;
    float part = 0.f;
    float* n = a.norm_state + ((size_t)slot * a.n_heads + h) * D;
    for (int d = tid; d < D; d += blockDim.x) {
      const float x = fmaf(keep, n[d], take * s_k[d]);      // (this thread's own s_k, s_q)
      n[d] = x;
      part = fmaf(x, s_q[d], part);
    }
    const float nq = block_sum(part, red) * a.q_scale;      // (also the barrier behind s_q and s_k)
    if (tid == 0) a.max_state[(size_t)slot * a.n_heads + h] = m;
    m = memory_size(nq, m);
  } else {
    for (int i = tid; i < a.rank; i += blockDim.x) {
      const float x = row[a.off_low + i];
      s_low[i] = a.decay_kind == DECAY_DOUBLE_EXP ? tanhf(x) : x;
    }
    __syncthreads();
    for (int d = tid; d < D; d += blockDim.x) {
      const int c = h * D + d;
      float z = a.bias ? a.bias[c] : 0.f;
      const float* w2 = a.w2 + (size_t)c * a.rank;
      if ((a.rank & 3) == 0) {
        for (int i = 0; i < a.rank; i += 4) {
          const floatx4 w4 = *(const floatx4*)(w2 + i);
#pragma unroll
          for (int q = 0; q < 4; ++q) z = fmaf(w4[q], s_low[i + q], z);
        }
      } else {
        for (int i = 0; i < a.rank; ++i) z = fmaf(w2[i], s_low[i], z);
      }
      s_a[d] = decay_of(z, a.decay_kind, a.inv_tau);
    }
    __syncthreads();
  }
  floatx4 acc = floatx4{0.f, 0.f, 0.f, 0.f};
  if (active) {
#pragma unroll
    for (int i = 0; i < ROWS; ++i) {
      const int d = g + a.groups * i;
      if (d < D) {
        const float k = s_k[d], q = s_q[d], decay = KIND == KIND_MEMORY ? keep : s_a[d];
        const float u = KIND == KIND_BONUS ? s_u[d] : 0.f;
#pragma unroll
        for (int c = 0; c < 4; ++c) {
          const float kv = k * v[c];
          if (KIND == KIND_BONUS) acc[c] = fmaf(fmaf(u, kv, S[i][c]), q, acc[c]);
          S[i][c] = fmaf(decay, S[i][c], kv);
          if (KIND != KIND_BONUS) acc[c] = fmaf(S[i][c], q, acc[c]);
        }
        *(floatx4*)(st + (size_t)d * E) = S[i];
      }
    }
#pragma unroll
    for (int c = 0; c < 4; ++c) s_sum[g * E + 4 * j + c] = acc[c];
  }
  __syncthreads();
  float o = 0.f;
  if (tid < E) {
    for (int i = 0; i < a.groups; ++i) o += s_sum[i * E + tid];
    o *= a.q_scale;
    if (KIND == KIND_MEMORY) o = o / m;
  }
  const float ms = block_sum(o * o, red) / (float)a.count;
  if (tid < E) {
    const float y = o * (1.0f / sqrtf(ms + a.eps)) * w;
    const float sg = 1.0f / (1.0f + expf(-gate));
    out[((size_t)r * a.n_heads + h) * E + tid] = from_float<T>(y * (a.gate_kind == 1 ? sg : gate * sg));
  }
}

constexpr int ROW_MAX_ROWS = 8;
// threads of a block (0: these sizes are not taken)
extern "C" int llmlab_recurrent_row_threads(int D, int E) {
  if (D <= 0 || E <= 0 || E % 4 != 0 || E > 1024 || D > 1024) return 0;
  for (int threads = (E + 63) / 64 * 64 < 256 ? 256 : (E + 63) / 64 * 64; threads <= 1024; threads += 64) {
    const int groups = threads / (E / 4);
    if ((D + groups - 1) / groups <= (threads < 512 ? 4 : ROW_MAX_ROWS)) return threads;
  }
  return 0;
}

extern "C" int llmlab_recurrent_row(const float* proj, int ld, int off_q, int off_k, int off_v, int off_g, float q_scale,
                                    int n_heads, int D, int E, float* state, const int* q_start, const int* req_rows,
                                    int n_reqs, const float* w, float eps, int w_per_head, int gate_kind, int norm_count,
                                    int kind, int off_low, int rank, const float* w2, const float* bias, int decay_kind,
                                    float tau, const float* bonus, int off_i, int off_f, const float* bias_i,
                                    const float* bias_f, float cap, float* norm_state, float* max_state, void* out, int dtype,
                                    hipStream_t stream) {
  const int threads = llmlab_recurrent_row_threads(D, E);
  LLMLAB_REQUIRE(threads > 0 && n_reqs >= 0 && n_heads > 0 && n_heads <= 65535, "recurrent_row: sizes D=%d E=%d heads=%d are not taken",
                 D, E, n_heads);
  LLMLAB_REQUIRE(proj && state && q_start && req_rows && w && out && norm_count >= 0 && norm_count <= E &&
                     (gate_kind == 0 || gate_kind == 1), "recurrent_row: an operand is missing");
  LLMLAB_REQUIRE(ld >= off_q + n_heads * D && ld >= off_k + n_heads * D && ld >= off_v + n_heads * E &&
                     ld >= off_g + n_heads * E && off_q >= 0 && off_k >= 0 && off_v >= 0 && off_g >= 0,
                 "recurrent_row: rows of %d numbers do not hold the projections", ld);
  LLMLAB_REQUIRE(kind >= KIND_DECAY && kind <= KIND_MEMORY, "recurrent_row: unknown kind %d", kind);
  if (kind == KIND_MEMORY) {
    LLMLAB_REQUIRE(norm_state && max_state && cap > 0.f && off_i >= 0 && off_f >= 0 && ld >= off_i + n_heads &&
                       ld >= off_f + n_heads, "recurrent_row: the memory's operands");
    rank = 0;
  } else {
    LLMLAB_REQUIRE(w2 && rank > 0 && rank <= ROW_MAX_RANK && off_low >= 0 && ld >= off_low + rank && tau > 0.f &&
                       (kind != KIND_BONUS || bonus), "recurrent_row: the decays' operands, a rank of up to %d", ROW_MAX_RANK);
  }
  if (n_reqs == 0) return 0;
  int groups = threads / (E / 4);
  if (groups > D) groups = D;
  const int rows = (D + groups - 1) / groups;
  const RowArgs a{proj, ld, off_q, off_k, off_v, off_g, q_scale, n_heads, D, E, groups, state, q_start, req_rows, w, eps,
                  w_per_head, gate_kind, norm_count > 0 ? norm_count : E, off_low, rank, w2, bias, decay_kind, 1.0f / tau,
                  bonus, off_i, off_f, bias_i, bias_f, cap, norm_state, max_state};
  const size_t lds = (size_t)(rank + 4 * D + groups * E) * sizeof(float);
  const dim3 grid(n_reqs, n_heads), block(threads);
#define LLMLAB_ROW(KIND, T, ROWS) \
  hipLaunchKernelGGL((recurrent_row_kernel<KIND, T, ROWS>), grid, block, lds, stream, a, (T*)out)
#define LLMLAB_ROW_ANY(KIND)                                    \
  do {                                                          \
    if (dtype == DT_BF16 && rows <= 4) LLMLAB_ROW(KIND, bf16_t, 4); \
    else if (dtype == DT_BF16) LLMLAB_ROW(KIND, bf16_t, ROW_MAX_ROWS); \
    else if (rows <= 4) LLMLAB_ROW(KIND, float, 4);             \
    else LLMLAB_ROW(KIND, float, ROW_MAX_ROWS);                 \
  } while (0)
  if (kind == KIND_DECAY) LLMLAB_ROW_ANY(KIND_DECAY);
  else if (kind == KIND_BONUS) LLMLAB_ROW_ANY(KIND_BONUS);
  else LLMLAB_ROW_ANY(KIND_MEMORY);
#undef LLMLAB_ROW_ANY
#undef LLMLAB_ROW
  LLMLAB_LAUNCH_CHECK("recurrent_row");
  return 0;
}


// ================================================================== generalised delta rule
// A matrix-valued state per head whose transition is a decay per key channel less a rank-one
// removal along the unit key, before the new key/value pair is written:
//   u_t = k_t / sqrt(|k_t|^2 + key_eps)
//   S_t = diag(w_t) S_(t-1) - (a_t * u_t) (u_t^T S_(t-1)) + k_t v_t^T        (decay and removal act on S_(t-1))
//   o_t = S_t^T r_t
// with w_t (decay) and a_t (removal rate) in (0, 1) per head and key channel.  State [D, E]
// per head, float32, one slot per request; everything here is float32.
//
// delta_gates, one block a row: w = exp(-decay_scale * sigmoid(w0 + W2 tanh(low))) from the
// low-rank projection `low` (rank numbers a row), a = sigmoid(a_in + a_bias), and what every
// column of the state needs of the row's key: the unit key u and the removal a * u.
constexpr int GATES_MAX_HEADS = 1024;
__global__ __launch_bounds__(256) void delta_gates_kernel(const float* __restrict__ proj, int ld, int off_low, int rank,
                                                          int off_a, int off_k, const float* __restrict__ w2,
                                                          const float* __restrict__ w0, const float* __restrict__ a_bias,
                                                          float decay_scale, float key_eps, float* __restrict__ decay,
                                                          float* __restrict__ unit, float* __restrict__ removal,
                                                          int n_heads, int D) {
  extern __shared__ float s_low[];       // tanh of the row's low-rank numbers, then 1 / |k| of every head
  float* s_inv = s_low + rank;
  const int r = blockIdx.x, channels = n_heads * D;
  const float* t = proj + (size_t)r * ld;
  for (int j = threadIdx.x; j < rank; j += blockDim.x) s_low[j] = tanhf(t[off_low + j]);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, waves = blockDim.x >> 6;
  for (int h = wave; h < n_heads; h += waves) {          // a wave a head
    float k2 = 0.f;
    for (int d = lane; d < D; d += 64) {
      const float k = t[off_k + h * D + d];
      k2 = fmaf(k, k, k2);
    }
    k2 = wave_sum(k2);
    if (lane == 0) s_inv[h] = 1.0f / sqrtf(k2 + key_eps);
  }
  __syncthreads();
  for (int c = threadIdx.x; c < channels; c += blockDim.x) {
    float z = w0 ? w0[c] : 0.f;
    const float* w = w2 + (size_t)c * rank;
    const float za = t[off_a + c] + (a_bias ? a_bias[c] : 0.f);
    const float u = t[off_k + c] * s_inv[c / D];
    if ((rank & 3) == 0) {                       // (a row of the second factor 16 bytes a load, all on their way together)
      for (int j = 0; j < rank; j += 4) {
        const floatx4 w4 = *(const floatx4*)(w + j);
        z = fmaf(w4[0], s_low[j], z);
        z = fmaf(w4[1], s_low[j + 1], z);
        z = fmaf(w4[2], s_low[j + 2], z);
        z = fmaf(w4[3], s_low[j + 3], z);
      }
    } else {
      for (int j = 0; j < rank; ++j) z = fmaf(w[j], s_low[j], z);
    }
    decay[(size_t)r * channels + c] = expf(-decay_scale / (1.0f + expf(-z)));
    unit[(size_t)r * channels + c] = u;
    removal[(size_t)r * channels + c] = u / (1.0f + expf(-za));
  }
}

extern "C" int llmlab_delta_gates(const float* proj, int ld, int rows, int off_low, int rank, int off_a, int off_k,
                                  const float* w2, const float* w0, const float* a_bias, float decay_scale,
                                  float key_eps, float* decay, float* unit, float* removal, int n_heads, int D,
                                  hipStream_t stream) {
  const int channels = n_heads * D;
  LLMLAB_REQUIRE(rows >= 0 && rank > 0 && rank <= 8192 && n_heads > 0 && n_heads <= GATES_MAX_HEADS && D > 0 &&
                 off_low >= 0 && off_a >= 0 && off_k >= 0 && ld >= off_low + rank && ld >= off_a + channels &&
                 ld >= off_k + channels,
                 "delta_gates: bad sizes rows=%d rank=%d heads=%d D=%d ld=%d", rows, rank, n_heads, D, ld);
  if (rows == 0) return 0;
  hipLaunchKernelGGL(delta_gates_kernel, dim3(rows), dim3(256), (rank + n_heads) * sizeof(float), stream, proj, ld,
                     off_low, rank, off_a, off_k, w2, w0, a_bias, decay_scale, key_eps, decay, unit, removal, n_heads, D);
  LLMLAB_LAUNCH_CHECK("delta_gates");
  return 0;
}

// delta_scan.  A quad of lanes keeps ONE column of a head's state in registers, a quarter of its
// DK >= D numbers each (the two sums over a column meet across the quad), and walks rows in order; the row's decay, unit key, removal, key and receptance are the same for
// every column: the block brings them into LDS a group of rows ahead (two buffers take turns, one
// barrier and one wait for memory a group), its value is one number a thread.  Per row and column: the dot product of the unit
// key with the column, the update, the dot product with the receptance.
//
// WHOLE: a block takes all the rows that a request brings to the step, for one head and 64
// columns: state from the request's slot and back.  Decode steps and short portions.
//
// Long portions are cut into chunks that run side by side, in three passes.  The recurrence is
// linear in the state, S_end = T S_start + L, with T (D x D) the product of the chunk's
// transitions diag(w) - (a * u) u^T and L the state the chunk builds from zero.  A column of T is
// what the recurrence without values makes of a unit vector, so:
//   LOCAL  per chunk: the E columns of L from zero and the D columns of T from the identity, no outputs;
//   carry  per request, chunk after chunk: S_start[c + 1] = T_c S_start[c] + L_c; the slot at the end;
//   FINISH per chunk: the rows again from S_start[c], now with outputs.
enum { DELTA_WHOLE = 0, DELTA_LOCAL = 1, DELTA_FINISH = 2 };

struct DeltaArgs {
  const float* proj; int ld, off_r, off_k, off_v;
  const float* decay; const float* unit; const float* removal;      // [rows, heads * D]
  int n_heads, D, E;
  float* state; const int* q_start; const int* req_rows; float* out;      // out [rows, heads, E]
  int n_reqs, chunk; float* chunk_state; float* chunk_trans;      // [chunks, heads, D, E] and [chunks, heads, D, D]
};

__device__ __forceinline__ bool delta_find_chunk(const DeltaArgs& a, int index, int& first, int& last) {
  int before = 0;
  for (int b = 0; b < a.n_reqs; ++b) {
    const int lo = a.q_start[b], hi = a.q_start[b + 1];
    const int n = (hi - lo + a.chunk - 1) / a.chunk;
    if (index < before + n) {
      first = lo + (index - before) * a.chunk;
      last = first + a.chunk < hi ? first + a.chunk : hi;
      return true;
    }
    before += n;
  }
  return false;
}

// the sum of a number over the four lanes of a quad (lanes 4 n .. 4 n + 3), in every one of them
__device__ __forceinline__ float quad_sum(float x) {
  x += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(x), 0xB1, 0xF, 0xF, true));      // lanes 1, 0, 3, 2
  x += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(x), 0x4E, 0xF, 0xF, true));      // lanes 2, 3, 0, 1
  return x;
}

template <int DK, int MODE>
__global__ __launch_bounds__(256) void delta_scan_kernel(DeltaArgs a) {
  constexpr int VECS = MODE == DELTA_LOCAL ? 4 : 5;      // decay, unit key, removal, key (, receptance)
  constexpr int DQ = DK / 4;                              // rows of a column that one lane of its quad keeps
  constexpr int PER = (VECS * DK + 255) / 256;            // numbers of a row that a thread brings
  constexpr int G = DK <= 64 ? 8 : (DK <= 128 ? 4 : 2);   // rows that travel together (one wait for memory per G rows)
  __shared__ __attribute__((aligned(16))) float tok[2][G][VECS][DK];
  const int h = blockIdx.y, D = a.D, E = a.E;
  const int q = threadIdx.x & 3, d0 = q * DQ;
  const int col = blockIdx.z * 64 + (int)(threadIdx.x >> 2);
  const int cols = MODE == DELTA_LOCAL ? E + D : E;
  int first, last;
  if (MODE == DELTA_WHOLE) {
    first = a.q_start[blockIdx.x];
    last = a.q_start[blockIdx.x + 1];
  } else if (!delta_find_chunk(a, blockIdx.x, first, last)) {
    return;
  }
  const bool live = col < cols;
  const bool is_value = col < E;                          // (LOCAL: the others are columns of the transition)
  const int e = is_value ? col : E - 1;
  float S[DQ];
  const float* s_in = MODE == DELTA_WHOLE ? a.state + ((size_t)a.req_rows[blockIdx.x] * a.n_heads + h) * D * E
                      : MODE == DELTA_FINISH ? a.chunk_state + ((size_t)blockIdx.x * a.n_heads + h) * D * E : nullptr;
#pragma unroll
  for (int i = 0; i < DQ; ++i) {
    const int d = d0 + i;
    if (MODE == DELTA_LOCAL) S[i] = (live && !is_value && d == col - E) ? 1.f : 0.f;
    else S[i] = (live && d < D) ? s_in[(size_t)d * E + e] : 0.f;
  }
  // the numbers of a row that this thread brings: number i of vector i / D, for i = tid, tid + 256, ...
  const int total = VECS * D;
  float pre[G][PER], v_pre[G], v_now[G];
  auto fetch = [&](int t0) {
#pragma unroll
    for (int g = 0; g < G; ++g) {
      if (g > 0 && t0 + g >= last) break;                          // (a decode step brings one row)
      const int t = t0 + g;
      const float* row = a.proj + (size_t)t * a.ld;
      const size_t at = ((size_t)t * a.n_heads + h) * D;
      v_pre[g] = is_value ? row[a.off_v + h * E + e] : 0.f;
#pragma unroll
      for (int n = 0; n < PER; ++n) {
        const int i = threadIdx.x + n * 256;
        float x = 0.f;
        if (i < total) {
          const int vec = i / D, d = i - vec * D;
          x = vec == 0 ? a.decay[at + d] : vec == 1 ? a.unit[at + d] : vec == 2 ? a.removal[at + d]
              : vec == 3 ? row[a.off_k + h * D + d] : row[a.off_r + h * D + d];
        }
        pre[g][n] = x;
      }
    }
  };
  auto stash = [&](int buf, int t0) {
#pragma unroll
    for (int g = 0; g < G; ++g) {
      if (g > 0 && t0 + g >= last) break;
#pragma unroll
      for (int n = 0; n < PER; ++n) {
        const int i = threadIdx.x + n * 256;
        if (i < total) {
          const int vec = i / D, d = i - vec * D;
          tok[buf][g][vec][d] = pre[g][n];
        }
      }
    }
  };
  // (vectors shorter than DK: the rest stays zero, so the sums over DK numbers need no bound)
  if (D < DK)
    for (int i = threadIdx.x; i < 2 * G * VECS * DK; i += 256) (&tok[0][0][0][0])[i] = 0.f;
  __syncthreads();
  if (first < last) {
    fetch(first);
    stash(0, first);
  }
  __syncthreads();
  for (int t0 = first, buf = 0; t0 < last; t0 += G, buf ^= 1) {
#pragma unroll
    for (int g = 0; g < G; ++g) v_now[g] = v_pre[g];
    const bool more = t0 + G < last;
    if (more) fetch(t0 + G);
#pragma unroll
    for (int g = 0; g < G; ++g) {
      const int t = t0 + g;
      if (t < last) {
        const float v = v_now[g];
        const float* w_ = &tok[buf][g][0][d0];
        const float* u_ = &tok[buf][g][1][d0];
        const float* au_ = &tok[buf][g][2][d0];
        const float* k_ = &tok[buf][g][3][d0];
        // (sums side by side, so that no sum waits for the one before it)
        float dots[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < DQ; ++i) dots[i & 3] = fmaf(u_[i], S[i], dots[i & 3]);
        const float dot = quad_sum((dots[0] + dots[1]) + (dots[2] + dots[3]));
        float os[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < DQ; ++i) {
          S[i] = fmaf(w_[i], S[i], fmaf(-au_[i], dot, k_[i] * v));
          if (MODE != DELTA_LOCAL) os[i & 3] = fmaf(S[i], tok[buf][g][VECS - 1][d0 + i], os[i & 3]);
        }
        if (MODE != DELTA_LOCAL) {
          const float o = quad_sum((os[0] + os[1]) + (os[2] + os[3]));
          if (live && q == 0) a.out[((size_t)t * a.n_heads + h) * E + e] = o;
        }
      }
    }
    if (more) stash(buf ^ 1, t0 + G);
    __syncthreads();
  }
  if (MODE == DELTA_FINISH || !live) return;
  float* dst;
  size_t stride;
  if (MODE == DELTA_WHOLE) {
    dst = a.state + ((size_t)a.req_rows[blockIdx.x] * a.n_heads + h) * D * E + e;
    stride = E;
  } else if (is_value) {
    dst = a.chunk_state + ((size_t)blockIdx.x * a.n_heads + h) * D * E + e;
    stride = E;
  } else {
    dst = a.chunk_trans + ((size_t)blockIdx.x * a.n_heads + h) * D * D + (col - E);
    stride = D;
  }
#pragma unroll
  for (int i = 0; i < DQ; ++i)
    if (d0 + i < D) dst[(size_t)(d0 + i) * stride] = S[i];
}

// carry: block (request, head, slab of 16 columns), CARRY_GROUPS waves; wave g computes the rows
// g, g + CARRY_GROUPS, ... of T_c S + L_c for the slab's columns: a column a quad of lanes, each lane
// a quarter of the sum over the old rows.  The slab of the state and the chunk's transition lie in
// LDS (a wave brings its own rows of the transition, the next chunk's while this chunk's sums are
// taken).  chunk_state[c] <- the state before chunk c.
constexpr int CARRY_GROUPS = 8, CARRY_COLS = 16;
template <int DK>
__global__ __launch_bounds__(64 * CARRY_GROUPS) void delta_carry_kernel(DeltaArgs a) {
  constexpr int ROWS = (DK + CARRY_GROUPS - 1) / CARRY_GROUPS, M = (DK + 63) / 64, DQ = DK / 4;
  __shared__ __attribute__((aligned(16))) float s_tr[ROWS * CARRY_GROUPS][DK + 4];
  __shared__ float s_col[DK][CARRY_COLS + 1];
  const int b = blockIdx.x, h = blockIdx.y, D = a.D, E = a.E;
  const int lane = threadIdx.x & 63, g = __builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6));
  const int q = lane & 3, c16 = lane >> 2, j0 = q * DQ;
  const int e = blockIdx.z * CARRY_COLS + c16;
  const bool live = e < E;
  const int ec = live ? e : E - 1;
  int before = 0;
  for (int r = 0; r < b; ++r) before += (a.q_start[r + 1] - a.q_start[r] + a.chunk - 1) / a.chunk;
  const int n = (a.q_start[b + 1] - a.q_start[b] + a.chunk - 1) / a.chunk;
  float* slot = a.state + ((size_t)a.req_rows[b] * a.n_heads + h) * D * E;
  for (int i = threadIdx.x; i < DK * CARRY_COLS; i += blockDim.x) {
    const int d = i / CARRY_COLS, c = i % CARRY_COLS;
    const int ee = blockIdx.z * CARRY_COLS + c;
    s_col[d][c] = (d < D && ee < E) ? slot[(size_t)d * E + ee] : 0.f;
  }
  // this wave's rows of a chunk's transition (64 entries of a row a register) and of its built state
  float tr[ROWS][M], built[ROWS];
  auto fetch = [&](int c) {
    const float* lp = a.chunk_state + ((size_t)c * a.n_heads + h) * D * E;
    const float* tp = a.chunk_trans + ((size_t)c * a.n_heads + h) * D * D;
#pragma unroll
    for (int i = 0; i < ROWS; ++i) {
      const int d = g + CARRY_GROUPS * i;
      built[i] = d < D ? lp[(size_t)d * E + ec] : 0.f;
#pragma unroll
      for (int m = 0; m < M; ++m) tr[i][m] = (d < D && 64 * m + lane < D) ? tp[(size_t)d * D + 64 * m + lane] : 0.f;
    }
  };
  auto stash = [&]() {
#pragma unroll
    for (int i = 0; i < ROWS; ++i)
#pragma unroll
      for (int m = 0; m < M; ++m)
        if (64 * m + lane < DK) s_tr[g + CARRY_GROUPS * i][64 * m + lane] = tr[i][m];
  };
  if (n > 0) {
    fetch(before);
    stash();
  }
  __syncthreads();
  for (int c = before; c < before + n; ++c) {
    float acc[ROWS];
#pragma unroll
    for (int i = 0; i < ROWS; ++i) acc[i] = q == 0 ? built[i] : 0.f;
    if (c + 1 < before + n) fetch(c + 1);                          // (on its way while the sums are taken)
    float* l = a.chunk_state + ((size_t)c * a.n_heads + h) * D * E;
#pragma unroll
    for (int jj = 0; jj < DQ; ++jj) {
      const float x = s_col[j0 + jj][c16];
#pragma unroll
      for (int i = 0; i < ROWS; ++i) acc[i] = fmaf(s_tr[g + CARRY_GROUPS * i][j0 + jj], x, acc[i]);
    }
#pragma unroll
    for (int i = 0; i < ROWS; ++i) acc[i] = quad_sum(acc[i]);
    if (live && q == 0) {                                          // the state before this chunk, in the chunk's place
#pragma unroll
      for (int i = 0; i < ROWS; ++i) {
        const int d = g + CARRY_GROUPS * i;
        if (d < D) l[(size_t)d * E + e] = s_col[d][c16];
      }
    }
    __syncthreads();                                               // (every wave has read the old columns and the transition)
    if (q == 0) {
#pragma unroll
      for (int i = 0; i < ROWS; ++i) {
        const int d = g + CARRY_GROUPS * i;
        if (d < DK) s_col[d][c16] = acc[i];
      }
    }
    if (c + 1 < before + n) stash();
    __syncthreads();
  }
  if (live && q == 0)
    for (int d = g; d < D; d += CARRY_GROUPS) slot[(size_t)d * E + e] = s_col[d][c16];
}

// proj [rows, ld] float32 holds r at off_r (heads * D), k at off_k, v at off_v (heads * E); decay,
// unit and removal [rows, heads * D] (delta_gates); state [slots, heads, D, E]; out [rows, heads, E].
// chunk > 0: the three-pass form over chunks of so many rows; chunk_state then holds max_chunks *
// heads * D * E floats and chunk_trans max_chunks * heads * D * D, max_chunks >= rows / chunk + n_reqs.
extern "C" int llmlab_delta_scan(const float* proj, int ld, int off_r, int off_k, int off_v, const float* decay,
                                 const float* unit, const float* removal, int n_heads, int D, int E, float* state,
                                 const int* q_start, const int* req_rows, int n_reqs, float* out, int rows, int chunk,
                                 float* chunk_state, float* chunk_trans, int max_chunks, hipStream_t stream) {
  LLMLAB_REQUIRE(rows >= 0 && n_reqs >= 0 && n_reqs <= 65535 && n_heads > 0 && n_heads <= 65535 && D > 0 && D <= 256 &&
                 E > 0 && E <= 16384,
                 "delta_scan: bad sizes rows=%d requests=%d heads=%d D=%d E=%d (keys up to 256 wide)", rows, n_reqs,
                 n_heads, D, E);
  LLMLAB_REQUIRE(off_r >= 0 && off_k >= 0 && off_v >= 0 && ld >= off_r + n_heads * D && ld >= off_k + n_heads * D &&
                 ld >= off_v + n_heads * E, "delta_scan: rows of %d numbers do not hold the projections", ld);
  if (rows == 0 || n_reqs == 0) return 0;
  DeltaArgs a{proj, ld, off_r, off_k, off_v, decay, unit, removal, n_heads, D, E, state, q_start, req_rows, out,
              n_reqs, chunk, chunk_state, chunk_trans};
#define LLMLAB_DELTA(DKV, MODE, GRIDX, COLS) \
  hipLaunchKernelGGL((delta_scan_kernel<DKV, MODE>), dim3(GRIDX, n_heads, ((COLS) + 63) / 64), dim3(256), 0, stream, a)
#define LLMLAB_DELTA_ANY(MODE, GRIDX, COLS)                   \
  do {                                                        \
    if (D <= 16) LLMLAB_DELTA(16, MODE, GRIDX, COLS);         \
    else if (D <= 32) LLMLAB_DELTA(32, MODE, GRIDX, COLS);    \
    else if (D <= 64) LLMLAB_DELTA(64, MODE, GRIDX, COLS);    \
    else if (D <= 128) LLMLAB_DELTA(128, MODE, GRIDX, COLS);  \
    else LLMLAB_DELTA(256, MODE, GRIDX, COLS);                \
  } while (0)
  LLMLAB_REQUIRE((E + 63) / 64 <= 65535 && (E + D + 63) / 64 <= 65535, "delta_scan: too many columns");
  if (chunk <= 0) {
    LLMLAB_DELTA_ANY(DELTA_WHOLE, n_reqs, E);
  } else {
    const int chunks = rows / chunk + n_reqs;
    LLMLAB_REQUIRE(chunk_state && chunk_trans && max_chunks >= chunks,
                   "delta_scan: %d rows of %d requests in chunks of %d need room for %d chunks, got %d", rows, n_reqs,
                   chunk, chunks, max_chunks);
    LLMLAB_REQUIRE(D <= 128, "delta_scan: chunks take states of up to 128 key channels, got %d", D);
    LLMLAB_DELTA_ANY(DELTA_LOCAL, chunks, E + D);
    const dim3 cgrid(n_reqs, n_heads, (E + CARRY_COLS - 1) / CARRY_COLS), cblock(64 * CARRY_GROUPS);
    if (D <= 16) hipLaunchKernelGGL(delta_carry_kernel<16>, cgrid, cblock, 0, stream, a);
    else if (D <= 32) hipLaunchKernelGGL(delta_carry_kernel<32>, cgrid, cblock, 0, stream, a);
    else if (D <= 64) hipLaunchKernelGGL(delta_carry_kernel<64>, cgrid, cblock, 0, stream, a);
    else hipLaunchKernelGGL(delta_carry_kernel<128>, cgrid, cblock, 0, stream, a);
    LLMLAB_DELTA_ANY(DELTA_FINISH, chunks, E);
  }
#undef LLMLAB_DELTA_ANY
#undef LLMLAB_DELTA
  LLMLAB_LAUNCH_CHECK("delta_scan");
  return 0;
}
