// A recurrence of single numbers, a channel by itself, whose gates are block-diagonal products, for gfx950:
//
//   u_t = conv_b + sum_j conv[j] x_(t - taps + 1 + j)          (channel by channel; nothing before the start)
//   r = sigmoid(R_p u_t + rb), i = sigmoid(I_p u_t + ib)       (p: the part of the channels; square matrices)
//   a = exp(c * r);  S_t = a S_(t-1) + sqrt(1 - a^2) i u_t;  out_t = S_t * gelu(y_t)
//
// x and y are float32 projections (biases added).  Everything is float32 but the operands of the gates'
// products, which are u and the matrices in the compute dtype (float32 on the matrix cores in true 32
// bits).  Channels are laid out in parts of `size` (a multiple of 32, zeros behind a part's own).
//
// Per request: S [channels] and the last inputs of the convolution in a ring [taps, channels], the input
// of position p at place p mod taps.  A step of one row writes a place that none of its readers read.
//
//   row      every request brings one row: convolution, gates, state and output in one launch
//   tiles    requests that bring many: tiles of 64 rows side by side.  First launch: convolution, gates,
//            and the recurrence within the tile from zero (the request's first tile: from its state) by
//            shifts between lanes; every row leaves the product of its tile's decays so far and the state
//            so far.  Second launch: the state a tile starts from, out of the last rows of the tiles before
//            it, folded into its rows; the request's last tile writes its slots.
#include "common.h"

extern "C" const char* llmlab_last_error() { return g_llmlab_error; }

constexpr int TILE_ROWS = 64;
template <typename T>                  // channels of a part that lie in LDS at a time
constexpr int SLAB = sizeof(T) == 4 ? 128 : 256;

template <typename T>
struct Recurrence {
  const float* proj; int ld, off_x, off_y;
  int channels, size;                  // channels = parts * size
  const float* conv; const float* conv_b; int taps;
  float* ring;
  const T* gates;                      // [part][strip of 16 outputs][32 inputs][R, I][lane][8]
  const float* rb; const float* ib; const float* c;
  float* state;
  const int* positions; const int* q_start; const int* req_rows; int n_reqs, rows;
  float* decays; float* states;        // [rows, channels]
  T* out;
};

template <typename T>
struct Eight { typedef bf16x8 V; };
template <>
struct Eight<float> { typedef __attribute__((__vector_size__(8 * sizeof(float)))) float V; };

// 16 outputs x 16 rows += 32 inputs: lane 16 g + c holds output c (weights) or row c (inputs) and the inputs
// 8 g .. 8 g + 7; the sums: row c, outputs 4 g .. 4 g + 3
__device__ __forceinline__ floatx4 multiply(bf16x8 w, bf16x8 u, floatx4 acc) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(w, u, acc, 0, 0, 0);
}
__device__ __forceinline__ floatx4 multiply(Eight<float>::V w, Eight<float>::V u, floatx4 acc) {
#pragma unroll
  for (int j = 0; j < 8; ++j) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(w[j], u[j], acc, 0, 0, 0);
  return acc;
}

// (reciprocal and square root to a unit in the last place, as the hardware gives them)
__device__ __forceinline__ float sigmoid_f(float z) { return __builtin_amdgcn_rcpf(1.0f + __expf(-z)); }
// tanh form of gelu, 0.5 z (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3))), as z * sigmoid(2 t)
__device__ __forceinline__ float gelu_f(float z) {
  return z * __builtin_amdgcn_rcpf(1.0f + __expf(-2.0f * 0.7978845608028654f * (z + 0.044715f * z * z * z)));
}
// sqrt(1 - a^2) for a = exp(l), l <= 0: near a = 1 by the series of 1 - exp(-y), y = -2 l (the sum of
// (-1)^k y^(k+1) / (k+1)!)
__device__ __forceinline__ float complement(float l, float a) {
  const float y = -2.0f * l;
  float s = 1.0f / 5040.0f;
  s = fmaf(s, y, -1.0f / 720.0f);
  s = fmaf(s, y, 1.0f / 120.0f);
  s = fmaf(s, y, -1.0f / 24.0f);
  s = fmaf(s, y, 1.0f / 6.0f);
  s = fmaf(s, y, -0.5f);
  s = fmaf(s, y, 1.0f);
  return __builtin_amdgcn_sqrtf(y < 0.35f ? y * s : fmaf(-a, a, 1.0f));
}

__device__ __forceinline__ floatx4 load4(const float* p) { return *(const floatx4*)p; }
__device__ __forceinline__ void store4(float* p, floatx4 v) { *(floatx4*)p = v; }
__device__ __forceinline__ void store4(bf16_t* p, floatx4 v) {
  *(bf16x4*)p = bf16x4{(bf16_t)v[0], (bf16_t)v[1], (bf16_t)v[2], (bf16_t)v[3]};
}

// The convolution at row r for the four channels from ch on; inside: rows of the request before r in the
// step; place: the ring's place of r's position; ring: the request's.  TAPS 0: any number.
template <typename T, int TAPS>
__device__ __forceinline__ floatx4 convolve(const Recurrence<T>& a, const float* ring, int r, int inside, int place, int ch) {
  const int taps = TAPS > 0 ? TAPS : a.taps;
  const float* x = a.proj + (size_t)r * a.ld + a.off_x + ch;
  floatx4 acc = load4(a.conv_b + ch);
  if (TAPS > 0) {
    floatx4 v[TAPS > 0 ? TAPS : 1], w[TAPS > 0 ? TAPS : 1];
#pragma unroll
    for (int k = 0; k < TAPS; ++k) {       // k positions back (the loads travel together)
      const int at = place - k < 0 ? place - k + TAPS : place - k;
      v[k] = load4(k <= inside ? x - (ptrdiff_t)k * a.ld : ring + (size_t)at * a.channels + ch);
      w[k] = load4(a.conv + (size_t)(TAPS - 1 - k) * a.channels + ch);
    }
#pragma unroll
    for (int k = TAPS - 1; k >= 0; --k) acc += w[k] * v[k];
  } else {
    for (int k = taps - 1; k >= 0; --k) {
      const int at = place - k < 0 ? place - k + taps : place - k;
      acc += load4(a.conv + (size_t)(taps - 1 - k) * a.channels + ch) *
             load4(k <= inside ? x - (ptrdiff_t)k * a.ld : ring + (size_t)at * a.channels + ch);
    }
  }
  return acc;
}

// ------------------------------------------------------------------ one row a request
// A block takes 16 * STRIPS outputs of a part and 16 rows (row r is request r); its four waves share the part's
// inputs, each making its operands from the projections and the rings itself.
template <typename T, int TAPS, int STRIPS>
__global__ __launch_bounds__(256) void recurrence_row_kernel(Recurrence<T> a) {
  typedef typename Eight<T>::V vec8;
  __shared__ floatx4 sums[4][STRIPS][2][64];
  const int lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int taps = TAPS > 0 ? TAPS : a.taps;
  const int strips = a.size >> 4, steps = a.size >> 5;
  const int strip0 = blockIdx.x * STRIPS, first = strip0 / strips * a.size;
  const int r0 = blockIdx.y * 16;
  // what the block's end needs, asked for first: a thread a row and an output of every strip
  const int er = min(r0 + (int)(threadIdx.x >> 4), a.rows - 1), ec = strip0 * 16 + (threadIdx.x & 15);
  const int e_slot = a.req_rows[er], e_place = a.positions[er] % taps;
  float* e_ring = taps > 1 ? a.ring + (size_t)e_slot * taps * a.channels + ec : nullptr;
  const float* e_row = a.proj + (size_t)er * a.ld + ec;
  float* s_at = a.state + (size_t)e_slot * a.channels + ec;
  float own[STRIPS], y[STRIPS], before[STRIPS], u[STRIPS], rb[STRIPS], ib[STRIPS], decay[STRIPS];
#pragma unroll
  for (int n = 0; n < STRIPS; ++n) {
    own[n] = e_row[a.off_x + 16 * n];
    y[n] = e_row[a.off_y + 16 * n];
    before[n] = s_at[16 * n];
    u[n] = a.conv_b[ec + 16 * n];
    rb[n] = a.rb[ec + 16 * n], ib[n] = a.ib[ec + 16 * n], decay[n] = a.c[ec + 16 * n];
  }
  for (int k = taps - 1; k > 0; --k) {
    const size_t at = (size_t)(e_place - k < 0 ? e_place - k + taps : e_place - k) * a.channels;
    const float* w = a.conv + (size_t)(taps - 1 - k) * a.channels + ec;
#pragma unroll
    for (int n = 0; n < STRIPS; ++n) u[n] = fmaf(w[16 * n], e_ring[at + 16 * n], u[n]);
  }
#pragma unroll
  for (int n = 0; n < STRIPS; ++n) u[n] = fmaf(a.conv[(size_t)(taps - 1) * a.channels + ec + 16 * n], own[n], u[n]);

  const int r = min(r0 + c, a.rows - 1);
  const float* ring = taps > 1 ? a.ring + (size_t)a.req_rows[r] * taps * a.channels : nullptr;
  const int place = a.positions[r] % taps;
  floatx4 acc[STRIPS][2];
#pragma unroll
  for (int n = 0; n < STRIPS; ++n) acc[n][0] = acc[n][1] = floatx4{0.f, 0.f, 0.f, 0.f};
  const vec8* w = (const vec8*)a.gates + (size_t)strip0 * steps * 128 + lane;
  for (int k = wave; k < steps; k += 4) {
    vec8 wr[STRIPS], wi[STRIPS];
#pragma unroll
    for (int n = 0; n < STRIPS; ++n) {
      wr[n] = w[((size_t)n * steps + k) * 128];
      wi[n] = w[((size_t)n * steps + k) * 128 + 64];
    }
    const int ch = first + 32 * k + 8 * g;
    const floatx4 lo = convolve<T, TAPS>(a, ring, r, 0, place, ch), hi = convolve<T, TAPS>(a, ring, r, 0, place, ch + 4);
    vec8 v;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      v[j] = from_float<T>(lo[j]);
      v[4 + j] = from_float<T>(hi[j]);
    }
#pragma unroll
    for (int n = 0; n < STRIPS; ++n) {
      acc[n][0] = multiply(wr[n], v, acc[n][0]);
      acc[n][1] = multiply(wi[n], v, acc[n][1]);
    }
  }
#pragma unroll
  for (int n = 0; n < STRIPS; ++n) {
    sums[wave][n][0][lane] = acc[n][0];
    sums[wave][n][1][lane] = acc[n][1];
  }
  __syncthreads();
  if (r0 + (int)(threadIdx.x >> 4) >= a.rows) return;
  const int from = 16 * ((threadIdx.x & 15) >> 2) + (threadIdx.x >> 4), q = threadIdx.x & 3;
#pragma unroll
  for (int n = 0; n < STRIPS; ++n) {
    float zr = rb[n], zi = ib[n];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      zr += sums[k][n][0][from][q];
      zi += sums[k][n][1][from][q];
    }
    const float l = decay[n] * sigmoid_f(zr), d = __expf(l);
    const float s = fmaf(d, before[n], complement(l, d) * sigmoid_f(zi) * u[n]);
    s_at[16 * n] = s;
    if (taps > 1) e_ring[(size_t)e_place * a.channels + 16 * n] = own[n];
    a.out[(size_t)er * a.channels + ec + 16 * n] = from_float<T>(s * gelu_f(y[n]));
  }
}

// ------------------------------------------------------------------ tiles of rows
struct Tile { int req, first, n, index; };      // the request, its first row and rows in the step, which of its tiles

// The tiles of 64 rows of the step's requests, in order; every wave finds its block's by itself.
__device__ __forceinline__ bool find_tile(const int* __restrict__ q_start, int n_reqs, int tile, Tile& t) {
  const int lane = threadIdx.x & 63;
  int before = 0;
  for (int b0 = 0; b0 < n_reqs; b0 += 64) {
    const int b = b0 + lane;
    const int first = b < n_reqs ? q_start[b] : 0, n = b < n_reqs ? q_start[b + 1] - first : 0;
    const int tiles = (n + TILE_ROWS - 1) / TILE_ROWS;
    int upto = tiles;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const int o = __shfl_up(upto, off, WAVE);
      upto += lane >= off ? o : 0;
    }
    const int all = __shfl(upto, 63, WAVE);
    if (tile < before + all) {
      const unsigned long long hit = __ballot(before + upto > tile);
      const int at = __builtin_ctzll(hit);
      t.req = __builtin_amdgcn_readfirstlane(b0 + at);
      t.first = __builtin_amdgcn_readfirstlane(__shfl(first, at, WAVE));
      t.n = __builtin_amdgcn_readfirstlane(__shfl(n, at, WAVE));
      t.index = __builtin_amdgcn_readfirstlane(tile - before - (__shfl(upto, at, WAVE) - __shfl(tiles, at, WAVE)));
      return true;
    }
    before += all;
  }
  return false;
}

// The steps S -> d S + s of four channels: of this lane and of all lanes before it within its row of 16,
// composed.  A lane takes the composed step of the lane 1, 2, 4, 8 before it in turn; lanes that have none
// keep theirs (a disabled lane of a shift is not written).  The wait in front: a shift reads a register two
// instructions after it was written at the earliest; within the block eight lie between.
#define LLMLAB_COMPOSE(N)                                                                       \
  "v_fmac_f32_dpp %4, %4, %0 row_shr:" #N " row_mask:0xf bank_mask:0xf\n"                       \
  "v_fmac_f32_dpp %5, %5, %1 row_shr:" #N " row_mask:0xf bank_mask:0xf\n"                       \
  "v_fmac_f32_dpp %6, %6, %2 row_shr:" #N " row_mask:0xf bank_mask:0xf\n"                       \
  "v_fmac_f32_dpp %7, %7, %3 row_shr:" #N " row_mask:0xf bank_mask:0xf\n"                       \
  "v_mul_f32_dpp %0, %0, %0 row_shr:" #N " row_mask:0xf bank_mask:0xf\n"                        \
  "v_mul_f32_dpp %1, %1, %1 row_shr:" #N " row_mask:0xf bank_mask:0xf\n"                        \
  "v_mul_f32_dpp %2, %2, %2 row_shr:" #N " row_mask:0xf bank_mask:0xf\n"                        \
  "v_mul_f32_dpp %3, %3, %3 row_shr:" #N " row_mask:0xf bank_mask:0xf\n"
__device__ __forceinline__ void compose(floatx4& d, floatx4& s) {
  float d0 = d[0], d1 = d[1], d2 = d[2], d3 = d[3], s0 = s[0], s1 = s[1], s2 = s[2], s3 = s[3];
  asm volatile("s_nop 1\n" LLMLAB_COMPOSE(1) LLMLAB_COMPOSE(2) LLMLAB_COMPOSE(4) LLMLAB_COMPOSE(8) "s_nop 1\n"
               : "+v"(d0), "+v"(d1), "+v"(d2), "+v"(d3), "+v"(s0), "+v"(s1), "+v"(s2), "+v"(s3));
  d = floatx4{d0, d1, d2, d3};
  s = floatx4{s0, s1, s2, s3};
}
#undef LLMLAB_COMPOSE

// the value of the last lane of the row of 16 lanes
__device__ __forceinline__ float last_of_16(float v) {
  return __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x15f, 0xf, 0xf, true));      // row_newbcast:15
}

// the value of the lane `n` before within the row of 16 lanes, round and round
template <int n>
__device__ __forceinline__ float lanes_round(float v) {
  return __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x120 + n, 0xf, 0xf, true));      // row_ror
}

// x[k] (k >= 1): the inputs k rows before this lane's, the rows of 16 lanes being consecutive rows `cur` and the
// 16 before them `prev`
template <int TAPS>
__device__ __forceinline__ void rows_back(const floatx4& prev, const floatx4& cur, int c, floatx4 (&x)[TAPS > 0 ? TAPS : 1]) {
  x[0] = cur;
#pragma unroll
  for (int q = 0; q < 4; ++q) {
    if constexpr (TAPS > 1) x[1][q] = lanes_round<1>(c >= 15 ? prev[q] : cur[q]);
    if constexpr (TAPS > 2) x[2][q] = lanes_round<2>(c >= 14 ? prev[q] : cur[q]);
    if constexpr (TAPS > 3) x[3][q] = lanes_round<3>(c >= 13 ? prev[q] : cur[q]);
  }
}

// A block takes a tile and, a strip a wave, up to blockDim.x / 4 outputs of a part.
template <typename T, int TAPS>
__global__ __launch_bounds__(512) __attribute__((amdgpu_waves_per_eu(4))) void recurrence_tiles_kernel(Recurrence<T> a) {
  typedef typename Eight<T>::V vec8;
  extern __shared__ __attribute__((aligned(16))) char tile_lds[];
  T* us = (T*)tile_lds;                           // [TILE_ROWS][slab + 8]
  Tile t;
  if (!find_tile(a.q_start, a.n_reqs, blockIdx.x, t)) return;
  const int lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int taps = TAPS > 0 ? TAPS : a.taps;
  const int threads = blockDim.x, waves = threads >> 6;
  const int strips = a.size >> 4, steps = a.size >> 5, groups = (strips + waves - 1) / waves;
  const int part = blockIdx.y / groups, strip = (blockIdx.y - part * groups) * waves + wave;
  const int first = part * a.size;
  const bool works = strip < strips;
  const int row0 = t.index * TILE_ROWS;           // within the request
  const int n = t.n - row0 < TILE_ROWS ? t.n - row0 : TILE_ROWS;
  const int slot = a.req_rows[t.req];
  const float* ring = taps > 1 ? a.ring + (size_t)slot * taps * a.channels : nullptr;
  const int pos0 = a.positions[t.first] + row0;   // of the tile's first row
  const int slab = a.size < SLAB<T> ? a.size : SLAB<T>, stride = slab + 8;
  // the input of row j of the request (negative: from before the step), four channels
  auto input = [&](int j, int ch) {
    const int place = j < 0 ? (pos0 - row0 + j + taps) % taps : 0;
    return load4(j >= 0 ? a.proj + ((unsigned)((t.first + j) * a.ld) + a.off_x + ch) : ring + (place * a.channels + ch));
  };
  floatx4 acc[4][2];
#pragma unroll
  for (int k = 0; k < 4; ++k) acc[k][0] = acc[k][1] = floatx4{0.f, 0.f, 0.f, 0.f};
  const vec8* w = (const vec8*)a.gates + ((size_t)part * strips + strip) * steps * 128 + lane;
  for (int k0 = 0; k0 < a.size; k0 += slab) {
    const int width = a.size - k0 < slab ? a.size - k0 : slab;
    if (k0) __syncthreads();                      // (the slab before has been read)
    // a thread four channels and a run of rows, the last inputs in registers
    const int quads = width >> 2, runs = threads / quads, run = (TILE_ROWS + runs - 1) / runs;
    const int q = threadIdx.x % quads, m0 = (int)threadIdx.x / quads * run, m1 = min(m0 + run, TILE_ROWS);
    const int ch = first + k0 + 4 * q;
    if constexpr (TAPS > 0) {
      floatx4 w[TAPS], x[TAPS], bias = load4(a.conv_b + ch);
      if (m0 < n) {
#pragma unroll
        for (int k = 0; k < TAPS; ++k) w[k] = load4(a.conv + (size_t)(TAPS - 1 - k) * a.channels + ch);
#pragma unroll
        for (int k = 1; k < TAPS; ++k) x[k] = input(row0 + m0 - k, ch);
      }
      for (int m = m0; m < m1; m += 4) {          // (four rows' loads travel together)
        floatx4 own[4];
        if (m < n)
#pragma unroll
          for (int i = 0; i < 4; ++i)
            own[i] = load4(a.proj + ((unsigned)((t.first + row0 + min(m + i, n - 1)) * a.ld) + a.off_x + ch));
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          if (m + i >= m1) break;
          floatx4 v = floatx4{0.f, 0.f, 0.f, 0.f};
          if (m + i < n) {
            x[0] = own[i];
            v = bias;
#pragma unroll
            for (int k = TAPS - 1; k >= 0; --k) v += w[k] * x[k];
#pragma unroll
            for (int k = TAPS - 1; k > 0; --k) x[k] = x[k - 1];
          }
          store4(us + (m + i) * stride + 4 * q, v);
        }
      }
    } else {
      for (int m = m0; m < m1; ++m) {
        floatx4 v = floatx4{0.f, 0.f, 0.f, 0.f};
        if (m < n) v = convolve<T, TAPS>(a, ring, t.first + row0 + m, row0 + m, (pos0 + m) % taps, ch);
        store4(us + m * stride + 4 * q, v);
      }
    }
    __syncthreads();
    if (works) {
      constexpr int AHEAD = sizeof(T) == 4 ? 2 : 4;       // steps whose matrices travel together
      const int count = width >> 5;
      for (int k1 = 0; k1 < count; k1 += AHEAD) {
        vec8 wr[AHEAD], wi[AHEAD];
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) {
          const int at = ((k0 >> 5) + min(k1 + i, count - 1)) * 128;
          wr[i] = w[at];
          wi[i] = w[at + 64];
        }
#pragma unroll
        for (int i = 0; i < AHEAD; ++i)
          if (k1 + i < count) {
#pragma unroll
            for (int m = 0; m < 4; ++m) {
              const vec8 v = *(const vec8*)(us + (16 * m + c) * stride + 32 * (k1 + i) + 8 * g);
              acc[m][0] = multiply(wr[i], v, acc[m][0]);
              acc[m][1] = multiply(wi[i], v, acc[m][1]);
            }
          }
      }
    }
  }
  if (!works) return;
  const int ch = first + 16 * strip + 4 * g;
  const floatx4 rb = load4(a.rb + ch), ib = load4(a.ib + ch), decay = load4(a.c + ch);
  floatx4 cw[TAPS > 0 ? TAPS : 1], cx[TAPS > 0 ? TAPS : 1], cb, prev, cur[4];
  if constexpr (TAPS > 0) {
    cb = load4(a.conv_b + ch);
#pragma unroll
    for (int k = 0; k < TAPS; ++k) cw[k] = load4(a.conv + (size_t)(TAPS - 1 - k) * a.channels + ch);
#pragma unroll
    for (int m = 0; m < 4; ++m)
      cur[m] = load4(a.proj + ((unsigned)((t.first + row0 + min(16 * m + c, n - 1)) * a.ld) + a.off_x + ch));
    prev = TAPS > 1 ? input(c > 16 - TAPS ? row0 + c - 16 : row0, ch) : cur[0];
  }
  floatx4 carry_d = floatx4{1.f, 1.f, 1.f, 1.f}, carry_s = floatx4{0.f, 0.f, 0.f, 0.f};
  if (t.index == 0) carry_s = load4(a.state + (size_t)slot * a.channels + ch);
#pragma unroll
  for (int m = 0; m < 4; ++m) {
    if (16 * m >= n) break;
    const int k = min(16 * m + c, n - 1);         // (lanes past the last row: that row again, not stored)
    const int r = t.first + row0 + k;
    floatx4 u;
    if constexpr (TAPS > 0) {
      rows_back<TAPS>(prev, cur[m], c, cx);
      prev = cur[m];
      u = cb;
#pragma unroll
      for (int j = TAPS - 1; j >= 0; --j) u += cw[j] * cx[j];
    } else {
      u = convolve<T, TAPS>(a, ring, r, row0 + k, (pos0 + k) % taps, ch);
    }
    floatx4 d, s;
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const float l = decay[q] * sigmoid_f(acc[m][0][q] + rb[q]);
      d[q] = __expf(l);
      s[q] = complement(l, d[q]) * sigmoid_f(acc[m][1][q] + ib[q]) * u[q];
    }
    compose(d, s);
    s += d * carry_s;
    d *= carry_d;
    if (16 * m + c < n) {
      store4(a.decays + (size_t)r * a.channels + ch, d);
      store4(a.states + (size_t)r * a.channels + ch, s);
    }
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      carry_d[q] = last_of_16(d[q]);
      carry_s[q] = last_of_16(s[q]);
    }
  }
}

// A block takes a tile and 256 channels, a lane four of them, a wave a run of the tile's rows, four at a time, of
// which it asks for the first four at once.  The waves compose the last rows of the tiles before theirs, a
// run of tiles a wave, and meet in LDS.
constexpr int CARRY_BATCH = 4;
template <typename T, int WAVES>
__global__ __launch_bounds__(64 * WAVES) void recurrence_carry_kernel(Recurrence<T> a) {
  constexpr int ROWS = TILE_ROWS / WAVES;
  __shared__ floatx4 run[WAVES][2][64];
  Tile t;
  if (!find_tile(a.q_start, a.n_reqs, blockIdx.x, t)) return;
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const bool mine = (int)blockIdx.y * 256 + 4 * lane < a.channels;
  const int ch = mine ? blockIdx.y * 256 + 4 * lane : 0;       // (lanes past the last channel: the first again, dropped)
  const int row0 = t.index * TILE_ROWS, lo = row0 + ROWS * wave;
  floatx4 d[CARRY_BATCH], s[CARRY_BATCH], y[CARRY_BATCH];
  auto ask = [&](int from) {
#pragma unroll
    for (int k = 0; k < CARRY_BATCH; ++k) {
      const int r = t.first + min(from + k, t.n - 1);
      d[k] = load4(a.decays + (size_t)r * a.channels + ch);
      s[k] = load4(a.states + (size_t)r * a.channels + ch);
      y[k] = load4(a.proj + (size_t)r * a.ld + a.off_y + ch);
    }
  };
  ask(lo);
  floatx4 start = floatx4{0.f, 0.f, 0.f, 0.f};
  if (t.index > 0) {                              // (the request's first tile has begun from its state)
    const int share = (t.index + WAVES - 1) / WAVES, first = wave * share, end = min(first + share, t.index);
    floatx4 dc = floatx4{1.f, 1.f, 1.f, 1.f}, sc = start;
#pragma unroll 4
    for (int k = first; k < end; ++k) {
      const size_t at = (size_t)(t.first + (k + 1) * TILE_ROWS - 1) * a.channels + ch;
      const floatx4 dk = load4(a.decays + at), sk = load4(a.states + at);
      sc = dk * sc + sk;
      dc *= dk;
    }
    run[wave][0][lane] = dc;
    run[wave][1][lane] = sc;
    __syncthreads();
#pragma unroll
    for (int k = 0; k < WAVES; ++k) start = run[k][0][lane] * start + run[k][1][lane];
  }
  if (!mine) return;
  const int slot = a.req_rows[t.req];
  for (int from = lo; from < lo + ROWS; from += CARRY_BATCH) {
    if (from > lo) ask(from);
#pragma unroll
    for (int k = 0; k < CARRY_BATCH; ++k) {
      if (from + k >= t.n) break;
      const floatx4 now = d[k] * start + s[k];
      floatx4 o;
#pragma unroll
      for (int q = 0; q < 4; ++q) o[q] = now[q] * gelu_f(y[k][q]);
      store4(a.out + (size_t)(t.first + from + k) * a.channels + ch, o);
      if (from + k == t.n - 1) store4(a.state + (size_t)slot * a.channels + ch, now);
    }
  }
  if (row0 + TILE_ROWS < t.n || a.taps <= 1) return;
  // the request's last tile, the ring: its last inputs (as many as it brought, at most one a place), a row a wave in turn
  const int pos0 = a.positions[t.first];
  float* ring = a.ring + (size_t)slot * a.taps * a.channels + ch;
  for (int k = t.n - 1 - wave; k >= 0 && k > t.n - 1 - a.taps; k -= WAVES)
    store4(ring + (size_t)((pos0 + k) % a.taps) * a.channels, load4(a.proj + (size_t)(t.first + k) * a.ld + a.off_x + ch));
}

template <typename T>
static int launch_recurrence(const Recurrence<T>& a, bool one_row_each, hipStream_t stream) {
  const int parts = a.channels / a.size, strips = a.size / 16;
#define LLMLAB_RECUR(KERNEL, GRID, THREADS, LDS, ...)                                                            \
  switch (a.taps) {                                                                                              \
    case 1: hipLaunchKernelGGL((KERNEL<T, 1 __VA_ARGS__>), GRID, dim3(THREADS), LDS, stream, a); break;          \
    case 2: hipLaunchKernelGGL((KERNEL<T, 2 __VA_ARGS__>), GRID, dim3(THREADS), LDS, stream, a); break;          \
    case 3: hipLaunchKernelGGL((KERNEL<T, 3 __VA_ARGS__>), GRID, dim3(THREADS), LDS, stream, a); break;          \
    case 4: hipLaunchKernelGGL((KERNEL<T, 4 __VA_ARGS__>), GRID, dim3(THREADS), LDS, stream, a); break;          \
    default: hipLaunchKernelGGL((KERNEL<T, 0 __VA_ARGS__>), GRID, dim3(THREADS), LDS, stream, a); break;         \
  }
  if (one_row_each) {
    // as many outputs a block as leave the chip its blocks: an operand made once serves them all (64 rows of
    // 3,584 channels in parts of 256: 15.6 us with 16 outputs a block)
    const int all = parts * strips, groups = (a.rows + 15) / 16;      // (a part has an even number of strips)
    if (strips % 4 == 0 && all / 4 * groups >= 192) {
      LLMLAB_RECUR(recurrence_row_kernel, dim3(all / 4, groups), 256, 0, , 4)
    } else if (all / 2 * groups >= 192) {
      LLMLAB_RECUR(recurrence_row_kernel, dim3(all / 2, groups), 256, 0, , 2)
    } else {
      LLMLAB_RECUR(recurrence_row_kernel, dim3(all, groups), 256, 0, , 1)
    }
    LLMLAB_LAUNCH_CHECK("gated_recurrence (one row a request)");
    return 0;
  }
  const int tiles = a.rows / TILE_ROWS + a.n_reqs;      // at most so many; blocks past the last leave at once
  const size_t lds = (size_t)TILE_ROWS * ((a.size < SLAB<T> ? a.size : SLAB<T>) + 8) * sizeof(T);
  // a part of 128 channels and more: eight waves a block, so that a block's inputs serve more outputs (2,048
  // rows of 3,584 channels in parts of 256, both launches: 68 us with four waves, 59 with eight)
  const int waves = strips >= 8 ? 8 : 4;
  const dim3 grid(tiles, parts * ((strips + waves - 1) / waves));
  LLMLAB_RECUR(recurrence_tiles_kernel, grid, 64 * waves, lds)
#undef LLMLAB_RECUR
  LLMLAB_LAUNCH_CHECK("gated_recurrence (tiles)");
  // few blocks: more waves a block (2,048 rows of 896 channels 13 us with four waves, 9 with sixteen; of 3,584
  // channels 19 and 24)
  const dim3 across(tiles, (a.channels + 255) / 256);
  if ((long)across.x * across.y <= 256)
    hipLaunchKernelGGL((recurrence_carry_kernel<T, 16>), across, dim3(1024), 0, stream, a);
  else
    hipLaunchKernelGGL((recurrence_carry_kernel<T, 4>), across, dim3(256), 0, stream, a);
  LLMLAB_LAUNCH_CHECK("gated_recurrence (carry)");
  return 0;
}


// proj [rows, ld] float32; gates and out in the compute dtype; q_start [n_reqs + 1]; decays, states (float32
// [rows, channels]): scratch of steps in which a request brings more than one row.
extern "C" int llmlab_gated_recurrence(const float* proj, int ld, int off_x, int off_y, int channels, int size,
                                       const float* conv, const float* conv_b, int taps, float* ring, const void* gates,
                                       const float* rb, const float* ib, const float* c, float* state,
                                       const int* positions, const int* q_start, const int* req_rows, int n_reqs, int rows,
                                       float* decays, float* states, void* out, int dtype, int one_row_each,
                                       hipStream_t stream) {
  LLMLAB_REQUIRE(rows >= 0 && size > 0 && size % 32 == 0 && channels > 0 && channels % size == 0 && taps >= 1,
                 "gated_recurrence: bad sizes rows=%d channels=%d size=%d taps=%d", rows, channels, size, taps);
  LLMLAB_REQUIRE(off_x >= 0 && off_y >= 0 && off_x % 4 == 0 && off_y % 4 == 0 && ld % 4 == 0 && off_x + channels <= ld &&
                     off_y + channels <= ld, "gated_recurrence: columns %d and %d of rows of %d numbers", off_x, off_y, ld);
  LLMLAB_REQUIRE(proj && conv && conv_b && gates && rb && ib && c && state && positions && q_start && req_rows && out &&
                     (taps == 1 || ring), "gated_recurrence: an operand is missing");
  LLMLAB_REQUIRE(one_row_each ? n_reqs == rows : (decays != nullptr && states != nullptr),
                 "gated_recurrence: %d rows of %d requests", rows, n_reqs);
  LLMLAB_REQUIRE((size_t)rows * ld < ((size_t)1 << 31), "gated_recurrence: %d rows of %d numbers", rows, ld);
  LLMLAB_REQUIRE(channels / 16 <= 65535 && rows / 16 <= 65535, "gated_recurrence: too many channels or rows");
  if (rows == 0 || n_reqs == 0) return 0;
  if (dtype == DT_BF16) {
    const Recurrence<bf16_t> a{proj, ld, off_x, off_y, channels, size, conv, conv_b, taps, ring, (const bf16_t*)gates, rb, ib,
                               c, state, positions, q_start, req_rows, n_reqs, rows, decays, states, (bf16_t*)out};
    return launch_recurrence(a, one_row_each != 0, stream);
  }
  const Recurrence<float> a{proj, ld, off_x, off_y, channels, size, conv, conv_b, taps, ring, (const float*)gates, rb, ib,
                            c, state, positions, q_start, req_rows, n_reqs, rows, decays, states, (float*)out};
  return launch_recurrence(a, one_row_each != 0, stream);
}
