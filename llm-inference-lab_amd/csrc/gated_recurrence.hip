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

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + __expf(-z)); }
// tanh form of gelu, 0.5 z (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3))), as z * sigmoid(2 t)
__device__ __forceinline__ float gelu_f(float z) {
  return z / (1.0f + __expf(-2.0f * 0.7978845608028654f * (z + 0.044715f * z * z * z)));
}
// sqrt(1 - a^2) for a = exp(l), l <= 0: near a = 1 by the series of 1 - exp(-y), y = -2 l
__device__ __forceinline__ float complement(float l, float a) {
  const float y = -2.0f * l;
  float s = 1.0f - y * (1.0f / 9.0f);
#pragma unroll
  for (int n = 8; n >= 2; --n) s = 1.0f - y * (1.0f / (float)n) * s;
  return sqrtf(y < 0.7f ? y * s : 1.0f - a * a);
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
// A block takes 16 outputs of a part and 16 rows (row r is request r); its four waves share the part's
// inputs, each making its operands from the projections and the rings itself.
template <typename T, int TAPS>
__global__ __launch_bounds__(256) void recurrence_row_kernel(Recurrence<T> a) {
  typedef typename Eight<T>::V vec8;
  __shared__ floatx4 sums[4][2][64];
  const int lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int taps = TAPS > 0 ? TAPS : a.taps;
  const int strips = a.size >> 4, steps = a.size >> 5;
  const int part = blockIdx.x / strips, first = part * a.size;
  const int r0 = blockIdx.y * 16;
  // what the block's end needs, asked for first: a thread a row and an output
  const int er = min(r0 + (int)(threadIdx.x >> 4), a.rows - 1), ec = blockIdx.x * 16 + (threadIdx.x & 15);
  const int e_slot = a.req_rows[er], e_place = a.positions[er] % taps;
  float* e_ring = taps > 1 ? a.ring + (size_t)e_slot * taps * a.channels + ec : nullptr;
  const float own = a.proj[(size_t)er * a.ld + a.off_x + ec];
  const float y = a.proj[(size_t)er * a.ld + a.off_y + ec];
  float* s_at = a.state + (size_t)e_slot * a.channels + ec;
  const float before = *s_at;
  float u = a.conv_b[ec];
  for (int k = taps - 1; k > 0; --k)
    u = fmaf(a.conv[(size_t)(taps - 1 - k) * a.channels + ec],
             e_ring[(size_t)(e_place - k < 0 ? e_place - k + taps : e_place - k) * a.channels], u);
  u = fmaf(a.conv[(size_t)(taps - 1) * a.channels + ec], own, u);
  const float rb = a.rb[ec], ib = a.ib[ec], decay = a.c[ec];

  const int r = min(r0 + c, a.rows - 1);
  const float* ring = taps > 1 ? a.ring + (size_t)a.req_rows[r] * taps * a.channels : nullptr;
  const int place = a.positions[r] % taps;
  floatx4 acc[2] = {floatx4{0.f, 0.f, 0.f, 0.f}, floatx4{0.f, 0.f, 0.f, 0.f}};
  const vec8* w = (const vec8*)a.gates + (size_t)blockIdx.x * steps * 128 + lane;
  for (int k = wave; k < steps; k += 4) {
    const vec8 wr = w[(size_t)k * 128], wi = w[(size_t)k * 128 + 64];
    const int ch = first + 32 * k + 8 * g;
    const floatx4 lo = convolve<T, TAPS>(a, ring, r, 0, place, ch), hi = convolve<T, TAPS>(a, ring, r, 0, place, ch + 4);
    vec8 v;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      v[j] = from_float<T>(lo[j]);
      v[4 + j] = from_float<T>(hi[j]);
    }
    acc[0] = multiply(wr, v, acc[0]);
    acc[1] = multiply(wi, v, acc[1]);
  }
  sums[wave][0][lane] = acc[0];
  sums[wave][1][lane] = acc[1];
  __syncthreads();
  const int from = 16 * ((threadIdx.x & 15) >> 2) + (threadIdx.x >> 4), q = threadIdx.x & 3;
  float zr = rb, zi = ib;
#pragma unroll
  for (int n = 0; n < 4; ++n) {
    zr += sums[n][0][from][q];
    zi += sums[n][1][from][q];
  }
  if (r0 + (int)(threadIdx.x >> 4) >= a.rows) return;
  const float l = decay * sigmoid_f(zr), d = __expf(l);
  const float s = fmaf(d, before, complement(l, d) * sigmoid_f(zi) * u);
  *s_at = s;
  if (taps > 1) e_ring[(size_t)e_place * a.channels] = own;
  a.out[(size_t)er * a.channels + ec] = from_float<T>(s * gelu_f(y));
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

// the value of the lane `n` before within the row of 16 lanes, `other` where there is none
template <int n>
__device__ __forceinline__ float lanes_back(float other, float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(__float_as_int(other), __float_as_int(v), 0x110 + n, 0xf, 0xf, false));
}

// The composed step (d, s): S -> d S + s of this lane and of all lanes before it within 16
template <int n>
__device__ __forceinline__ void compose(float& d, float& s) {
  const float pd = lanes_back<n>(1.f, d), ps = lanes_back<n>(0.f, s);
  s = fmaf(d, ps, s);
  d *= pd;
}

template <typename T, int TAPS>
__global__ __launch_bounds__(256) void recurrence_tiles_kernel(Recurrence<T> a) {
  typedef typename Eight<T>::V vec8;
  extern __shared__ __attribute__((aligned(16))) char tile_lds[];
  T* us = (T*)tile_lds;                           // [TILE_ROWS][slab + 8]
  Tile t;
  if (!find_tile(a.q_start, a.n_reqs, blockIdx.x, t)) return;
  const int lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int taps = TAPS > 0 ? TAPS : a.taps;
  const int strips = a.size >> 4, steps = a.size >> 5, groups = (strips + 3) >> 2;
  const int part = blockIdx.y / groups, strip = (blockIdx.y - part * groups) * 4 + wave;
  const int first = part * a.size;
  const bool works = strip < strips;
  const int row0 = t.index * TILE_ROWS;           // within the request
  const int n = t.n - row0 < TILE_ROWS ? t.n - row0 : TILE_ROWS;
  const int slot = a.req_rows[t.req];
  const float* ring = taps > 1 ? a.ring + (size_t)slot * taps * a.channels : nullptr;
  const int pos0 = a.positions[t.first] + row0;   // of the tile's first row
  const int slab = a.size < SLAB<T> ? a.size : SLAB<T>, stride = slab + 8;
  floatx4 acc[4][2];
#pragma unroll
  for (int k = 0; k < 4; ++k) acc[k][0] = acc[k][1] = floatx4{0.f, 0.f, 0.f, 0.f};
  const vec8* w = (const vec8*)a.gates + ((size_t)part * strips + strip) * steps * 128 + lane;
  for (int k0 = 0; k0 < a.size; k0 += slab) {
    const int width = a.size - k0 < slab ? a.size - k0 : slab;
    if (k0) __syncthreads();                      // (the slab before has been read)
    // a thread four channels and every so many rows
    const int quads = width >> 2, apart = 256 / quads;
    const int q = threadIdx.x % quads;
    for (int m = threadIdx.x / quads; m < TILE_ROWS && (int)threadIdx.x < quads * apart; m += apart) {
      floatx4 v = floatx4{0.f, 0.f, 0.f, 0.f};
      if (m < n) v = convolve<T, TAPS>(a, ring, t.first + row0 + m, row0 + m, (pos0 + m) % taps, first + k0 + 4 * q);
      store4(us + m * stride + 4 * q, v);
    }
    __syncthreads();
    if (works)
      for (int k = 0; k < width >> 5; ++k) {
        const size_t at = (size_t)((k0 >> 5) + k) * 128;
        const vec8 wr = w[at], wi = w[at + 64];
#pragma unroll
        for (int m = 0; m < 4; ++m) {
          const vec8 v = *(const vec8*)(us + (16 * m + c) * stride + 32 * k + 8 * g);
          acc[m][0] = multiply(wr, v, acc[m][0]);
          acc[m][1] = multiply(wi, v, acc[m][1]);
        }
      }
  }
  if (!works) return;
  const int ch = first + 16 * strip + 4 * g;
  const floatx4 rb = load4(a.rb + ch), ib = load4(a.ib + ch), decay = load4(a.c + ch);
  floatx4 carry_d = floatx4{1.f, 1.f, 1.f, 1.f}, carry_s = floatx4{0.f, 0.f, 0.f, 0.f};
  if (t.index == 0) carry_s = load4(a.state + (size_t)slot * a.channels + ch);
#pragma unroll
  for (int m = 0; m < 4; ++m) {
    if (16 * m >= n) break;
    const int k = min(16 * m + c, n - 1);         // (lanes past the last row: that row again, not stored)
    const int r = t.first + row0 + k;
    const floatx4 u = convolve<T, TAPS>(a, ring, r, row0 + k, (pos0 + k) % taps, ch);
    floatx4 d, s;
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const float l = decay[q] * sigmoid_f(acc[m][0][q] + rb[q]);
      d[q] = __expf(l);
      s[q] = complement(l, d[q]) * sigmoid_f(acc[m][1][q] + ib[q]) * u[q];
      float dq = d[q], sq = s[q];
      compose<1>(dq, sq);
      compose<2>(dq, sq);
      compose<4>(dq, sq);
      compose<8>(dq, sq);
      s[q] = fmaf(dq, carry_s[q], sq);
      d[q] = dq * carry_d[q];
    }
    if (16 * m + c < n) {
      store4(a.decays + (size_t)r * a.channels + ch, d);
      store4(a.states + (size_t)r * a.channels + ch, s);
    }
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      carry_d[q] = __shfl(d[q], (lane & 48) + 15, WAVE);
      carry_s[q] = __shfl(s[q], (lane & 48) + 15, WAVE);
    }
  }
}

// A block takes a tile and 256 channels, a lane four of them.  The waves compose the last rows of the tiles
// before theirs, a run of tiles a wave, and meet in LDS; then each takes 16 of the tile's rows.
template <typename T>
__global__ __launch_bounds__(256) void recurrence_carry_kernel(Recurrence<T> a) {
  __shared__ floatx4 run[4][2][64];
  Tile t;
  if (!find_tile(a.q_start, a.n_reqs, blockIdx.x, t)) return;
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int ch = blockIdx.y * 256 + 4 * lane;
  const bool mine = ch < a.channels;
  floatx4 start = floatx4{0.f, 0.f, 0.f, 0.f};
  if (t.index > 0) {                              // (the request's first tile has begun from its state)
    const int share = (t.index + 3) >> 2, lo = wave * share, hi = min(lo + share, t.index);
    floatx4 d = floatx4{1.f, 1.f, 1.f, 1.f}, s = start;
    if (mine)
      for (int k = lo; k < hi; ++k) {
        const size_t at = (size_t)(t.first + (k + 1) * TILE_ROWS - 1) * a.channels + ch;
        const floatx4 dk = load4(a.decays + at), sk = load4(a.states + at);
        s = dk * s + sk;
        d *= dk;
      }
    run[wave][0][lane] = d;
    run[wave][1][lane] = s;
    __syncthreads();
#pragma unroll
    for (int k = 0; k < 4; ++k) start = run[k][0][lane] * start + run[k][1][lane];
  }
  if (!mine) return;
  const int slot = a.req_rows[t.req];
  const int row0 = t.index * TILE_ROWS;
  const bool last_tile = row0 + TILE_ROWS >= t.n;
  const int lo = row0 + 16 * wave, hi = min(lo + 16, t.n);
#pragma unroll 4
  for (int k = lo; k < hi; ++k) {
    const size_t r = (size_t)(t.first + k), at = r * a.channels + ch;
    const floatx4 s = load4(a.decays + at) * start + load4(a.states + at);
    const floatx4 y = load4(a.proj + r * a.ld + a.off_y + ch);
    floatx4 o;
#pragma unroll
    for (int q = 0; q < 4; ++q) o[q] = s[q] * gelu_f(y[q]);
    store4(a.out + at, o);
    if (k == t.n - 1) store4(a.state + (size_t)slot * a.channels + ch, s);
  }
  if (!last_tile || a.taps <= 1) return;
  // the ring: the request's last inputs (as many as it brought, at most one a place), a wave every fourth
  const int pos0 = a.positions[t.first];
  float* ring = a.ring + (size_t)slot * a.taps * a.channels + ch;
  for (int k = t.n - 1 - wave; k >= 0 && k > t.n - 1 - a.taps; k -= 4)
    store4(ring + (size_t)((pos0 + k) % a.taps) * a.channels, load4(a.proj + (size_t)(t.first + k) * a.ld + a.off_x + ch));
}

template <typename T>
static int launch_recurrence(const Recurrence<T>& a, bool one_row_each, hipStream_t stream) {
  const int parts = a.channels / a.size, strips = a.size / 16;
#define LLMLAB_RECUR(KERNEL, GRID, LDS)                                                                          \
  switch (a.taps) {                                                                                              \
    case 1: hipLaunchKernelGGL((KERNEL<T, 1>), GRID, dim3(256), LDS, stream, a); break;                          \
    case 2: hipLaunchKernelGGL((KERNEL<T, 2>), GRID, dim3(256), LDS, stream, a); break;                          \
    case 3: hipLaunchKernelGGL((KERNEL<T, 3>), GRID, dim3(256), LDS, stream, a); break;                          \
    case 4: hipLaunchKernelGGL((KERNEL<T, 4>), GRID, dim3(256), LDS, stream, a); break;                          \
    default: hipLaunchKernelGGL((KERNEL<T, 0>), GRID, dim3(256), LDS, stream, a); break;                         \
  }
  if (one_row_each) {
    const dim3 grid(parts * strips, (a.rows + 15) / 16);
    LLMLAB_RECUR(recurrence_row_kernel, grid, 0)
    LLMLAB_LAUNCH_CHECK("gated_recurrence (one row a request)");
    return 0;
  }
  const int tiles = a.rows / TILE_ROWS + a.n_reqs;      // at most so many; blocks past the last leave at once
  const size_t lds = (size_t)TILE_ROWS * ((a.size < SLAB<T> ? a.size : SLAB<T>) + 8) * sizeof(T);
  const dim3 grid(tiles, parts * ((strips + 3) / 4));
  LLMLAB_RECUR(recurrence_tiles_kernel, grid, lds)
#undef LLMLAB_RECUR
  LLMLAB_LAUNCH_CHECK("gated_recurrence (tiles)");
  hipLaunchKernelGGL(recurrence_carry_kernel<T>, dim3(tiles, (a.channels + 255) / 256), dim3(256), 0, stream, a);
  LLMLAB_LAUNCH_CHECK("gated_recurrence (carry)");
  return 0;
}

extern "C" int llmlab_gated_recurrence_tile_rows() { return TILE_ROWS; }

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
