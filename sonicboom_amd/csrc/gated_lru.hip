// A real-gated linear recurrence behind a short convolution, channel by channel, with gates that are products within
// equal blocks of channels:
//     u_t = sum_j w[c][j] x_(t - taps + 1 + j) + bw[c],  x = the input product + bx   (zeros before the sequence)
//     r = sigmoid(Ra u_b + ba), i = sigmoid(Ri u_b + bi)      in every block b of m channels (Ra, Ri m x m)
//     log a = -rate[c] r,  S_t = a S_(t-1) + sqrt(1 - a^2) i u,  out_t = S_t gelu(y_t + by)
// All of it in float32.  A sequence's state is S [width] and the last `taps` inputs of the convolution, kept by position:
// the input of position p lies in row p % taps, so a step reads the rows of earlier positions and writes others.
//
// Forms:
//   step     every sequence brings one row: one launch.  A block holds up to eight rows' u of one block of channels in
//            LDS and works out sixteen channels: sixteen lanes a channel share its two products.
//   walk     any rows: the same kernel leaves (a, sqrt(1 - a^2) i u) of every row, then a thread a channel walks the rows.
//            A row's numbers are worked out by the same operations in the same order as in the step form.
//   chunked  runs of up to 64 consecutive rows of one sequence, for prompts in bfloat16: the products on the matrix cores
//            with u as the sum of three bfloat16 numbers (all of its 24 bits; the weights are bfloat16, so every product
//            is exact and the sums are float32), the pair folded over the run; then the state carried from run to run;
//            then every run walked in four parts at once, each from the state that its place in the run gives.
#include "mfma.h"

namespace {

constexpr int kMaxTaps = 16;
constexpr int kChunk = 64, kPart = 16;
constexpr int kRows = 8;               // rows a block of the step form takes
constexpr int kMaxBlock = 1536;        // channels of a block: kRows of them lie in LDS
constexpr int kMaxBlockMfma = 256;

struct LruArgs {
  void *out; int out_dtype;                                      // [rows, width]
  const float *x, *y; int row_stride, n_slices; size_t slice_stride;
  const float *x_bias, *y_bias;                                  // [width]
  const float *taps_w, *taps_b; int taps;                        // [width, taps], [width]
  const void *ra, *ri; int w_dtype;                              // [width / m, m, m]: [out][in]
  const float *ra_b, *ri_b, *rate;                               // [width]
  float *state, *ring;                                           // [slots, width], [slots, taps, width]
  const int32_t *row_pos, *row_seq, *cu_rows, *slots;
  int n_rows, n_seqs, width, m;
  float2 *ab;                                                    // [rows, width]
  const int32_t *chunks; int n_chunks; float2 *folded;           // [n_chunks, width]
};

constexpr float kLog2e = 1.4426950408889634f;

// By the hardware's exponential, reciprocal and root (a unit or two of the last digit each); an exponential's argument is
// rounded once more on its way to base two, which counts as much as the rounding of the argument itself.
__device__ __forceinline__ float exp_f(float v) { return __builtin_amdgcn_exp2f(v * kLog2e); }
__device__ __forceinline__ float sigmoid_f(float v) { return __builtin_amdgcn_rcpf(1.0f + exp_f(-v)); }

// (1 + tanh x) / 2 = sigmoid(2 x)
__device__ __forceinline__ float gelu_f(float g) { return g * sigmoid_f(1.5957691216057308f * g * fmaf(0.044715f * g, g, 1.0f)); }

// 1 - exp(-y) for y >= 0 with e = exp(-y) at hand: the series below y = 1/2 (its next term is below the last digit there)
__device__ __forceinline__ float one_minus_exp(float y, float e) {
  float p = fmaf(y, -1.0f / 8.0f, 1.0f);
  p = fmaf(y * (-1.0f / 7.0f), p, 1.0f);
  p = fmaf(y * (-1.0f / 6.0f), p, 1.0f);
  p = fmaf(y * (-1.0f / 5.0f), p, 1.0f);
  p = fmaf(y * (-1.0f / 4.0f), p, 1.0f);
  p = fmaf(y * (-1.0f / 3.0f), p, 1.0f);
  p = fmaf(y * (-1.0f / 2.0f), p, 1.0f);
  return y < 0.5f ? y * p : 1.0f - e;
}

__device__ __forceinline__ float input_at(const LruArgs &a, int row, int c) {
  return sum_slices(a.x + size_t(row) * a.row_stride + c, a.n_slices, a.slice_stride) + a.x_bias[c];
}

// The convolution's input `back` rows before row r of the sequence (its row `row` of the step, at position pos).
__device__ __forceinline__ float input_back(const LruArgs &a, int row, int r, int pos, int slot, int back, int c) {
  if (back <= r) return input_at(a, row - back, c);
  const float kept = a.ring[(size_t(slot) * a.taps + max(pos - back, 0) % a.taps) * a.width + c];
  return pos < back ? 0.0f : kept;
}

// u of a row.  T: the taps where the kernel is compiled for their number, or 0.
template <int T>
__device__ __forceinline__ float conv_at(const LruArgs &a, int row, int r, int pos, int slot, int c, float &current) {
  float acc = 0.0f;
  if (T > 0) {
    float in[T > 0 ? T : 1];
#pragma unroll
    for (int j = 0; j < T; ++j) in[j] = input_back(a, row, r, pos, slot, T - 1 - j, c);
#pragma unroll
    for (int j = 0; j < T; ++j) acc = fmaf(a.taps_w[size_t(c) * T + j], in[j], acc);
    current = in[T > 0 ? T - 1 : 0];
  } else {
    for (int j = 0; j < a.taps; ++j) {
      current = input_back(a, row, r, pos, slot, a.taps - 1 - j, c);
      acc = fmaf(a.taps_w[size_t(c) * a.taps + j], current, acc);
    }
  }
  return acc + a.taps_b[c];
}

__device__ __forceinline__ float2 decay_and_input(float zr, float zi, float u, float rate) {
  const float r = sigmoid_f(zr), i = sigmoid_f(zi), y = rate * r, a = exp_f(-y);
  return make_float2(a, __builtin_amdgcn_sqrtf(one_minus_exp(2.0f * y, a * a)) * (i * u));
}

__device__ __forceinline__ void store_out(const LruArgs &a, int row, int c, float S, float y) {
  const float o = S * gelu_f(y);
  if (a.out_dtype == SB_F32) ((float *)a.out)[size_t(row) * a.width + c] = o;
  else ((bf16_t *)a.out)[size_t(row) * a.width + c] = f32_to_bf16(o);
}

__device__ __forceinline__ void load8(const float *p, float (&v)[8]) {
  const float4 a = reinterpret_cast<const float4 *>(p)[0], b = reinterpret_cast<const float4 *>(p)[1];
  v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
}

// Eight neighbouring weights as they lie in memory.
struct Eight16 { uint4 v; };
struct Eight32 { float4 a, b; };
template <typename TW> struct RawOf;
template <> struct RawOf<bf16_t> { typedef Eight16 type; };
template <> struct RawOf<float> { typedef Eight32 type; };
__device__ __forceinline__ void raw8(Eight16 &r, const bf16_t *p) { r.v = *reinterpret_cast<const uint4 *>(p); }
__device__ __forceinline__ void raw8(Eight32 &r, const float *p) {
  r.a = reinterpret_cast<const float4 *>(p)[0];
  r.b = reinterpret_cast<const float4 *>(p)[1];
}
__device__ __forceinline__ void unpack8(const Eight16 &r, float (&v)[8]) {
  const uint32_t u[4] = {r.v.x, r.v.y, r.v.z, r.v.w};
#pragma unroll
  for (int i = 0; i < 4; ++i) { v[2 * i] = __uint_as_float(u[i] << 16); v[2 * i + 1] = __uint_as_float(u[i] & 0xffff0000u); }
}
__device__ __forceinline__ void unpack8(const Eight32 &r, float (&v)[8]) {
  v[0] = r.a.x; v[1] = r.a.y; v[2] = r.a.z; v[3] = r.a.w; v[4] = r.b.x; v[5] = r.b.y; v[6] = r.b.z; v[7] = r.b.w;
}

// grid (blocks of channels * sixteens of a block, rows / kRows).  In a step row i is sequence i's only one: what the kernel
// needs from memory is asked for in two rounds (the rows' positions and slots with the weights, then everything that hangs
// on them).  SL: 1 for whole rows, 8 for rows in up to eight K slices, 0 for any number.
template <typename TW, int T, bool STEP, int SL>
__global__ void __launch_bounds__(256) lru_gates_kernel(LruArgs a, int vec) {
  extern __shared__ __attribute__((aligned(16))) float us[];         // [kRows][padded]
  __shared__ int pos_of[kRows], slot_of[kRows];
  const int padded = (a.m + 7) & ~7, per_block = (a.m + 15) / 16;
  const int blk = blockIdx.x / per_block, o0 = (blockIdx.x % per_block) * 16, c0 = blk * a.m;
  const int row0 = blockIdx.y * kRows, nr = min(kRows, a.n_rows - row0), tid = threadIdx.x;
  const int lane16 = tid & 15, o = o0 + (tid >> 4);
  const bool live = o < a.m;
  const int c = c0 + min(o, a.m - 1);
  const int my_row = row0 + min(lane16, nr - 1);
  const TW *wr = (const TW *)a.ra + size_t(c) * a.m, *wi = (const TW *)a.ri + size_t(c) * a.m;
  if (tid < kRows) {
    const int row = row0 + min(tid, nr - 1);
    pos_of[tid] = a.row_pos[row];
    slot_of[tid] = a.slots[STEP ? row : a.row_seq[row]];
  }
  typename RawOf<TW>::type raw_r, raw_i;
  if (vec) {
    const int k = min(8 * lane16, a.m - 8);        // (lanes past the block's end do not use them)
    raw8(raw_r, wr + k);
    raw8(raw_i, wi + k);
  }
  const float br = a.ra_b[c], bi = a.ri_b[c], rate = a.rate[c];
  __syncthreads();
  float S = 0.0f, y_in[SL > 0 ? SL : 1];
  const int my_slot = slot_of[lane16 & (kRows - 1)];
  if (STEP) {
    S = a.state[size_t(my_slot) * a.width + c];
    if (SL > 0)
#pragma unroll
      for (int s = 0; s < SL; ++s) y_in[s] = a.y[min(s, a.n_slices - 1) * a.slice_stride + size_t(my_row) * a.row_stride + c];
  }
  if constexpr (STEP && T > 0 && SL > 0) {
    constexpr int U = 4;                            // numbers of u that a thread works on at once
    for (int base = tid; base < kRows * padded; base += 256 * U) {
      float x_in[U][SL], kept[U][T];                // kept[j][t]: the input T - 1 - t rows back
      float w[U][T], bx[U], bw[U];
#pragma unroll
      for (int j = 0; j < U; ++j) {
        const int idx = min(base + 256 * j, kRows * padded - 1), i = idx / padded, k = min(idx - i * padded, a.m - 1);
        const int row = row0 + min(i, nr - 1), pos = pos_of[i];
        const float *ring = a.ring + size_t(slot_of[i]) * T * a.width + c0 + k;
#pragma unroll
        for (int s = 0; s < SL; ++s) x_in[j][s] = a.x[min(s, a.n_slices - 1) * a.slice_stride + size_t(row) * a.row_stride + c0 + k];
#pragma unroll
        for (int t = 0; t < T - 1; ++t) kept[j][t] = ring[size_t(max(pos - (T - 1 - t), 0) % T) * a.width];
#pragma unroll
        for (int t = 0; t < T; ++t) w[j][t] = a.taps_w[size_t(c0 + k) * T + t];
        bx[j] = a.x_bias[c0 + k];
        bw[j] = a.taps_b[c0 + k];
      }
#pragma unroll
      for (int j = 0; j < U; ++j) {
        const int idx = base + 256 * j, i = idx / padded, k = idx - i * padded;
        if (idx >= kRows * padded) continue;
        const bool on = i < nr && k < a.m;
        const int pos = pos_of[min(i, kRows - 1)];
        float cur = x_in[j][0];
#pragma unroll
        for (int s = 1; s < SL; ++s)
          if (s < a.n_slices) cur += x_in[j][s];
        cur += bx[j];
        float acc = 0.0f;
#pragma unroll
        for (int t = 0; t < T - 1; ++t) acc = fmaf(w[j][t], pos < T - 1 - t ? 0.0f : kept[j][t], acc);
        acc = fmaf(w[j][T - 1], cur, acc) + bw[j];
        if (on && k >= o0 && k < o0 + 16) a.ring[(size_t(slot_of[i]) * T + pos % T) * a.width + c0 + k] = cur;
        us[idx] = on ? acc : 0.0f;
      }
    }
  } else {
    for (int idx = tid; idx < kRows * padded; idx += 256) {
      const int i = idx / padded, k = idx - i * padded;
      float u = 0.0f;
      if (i < nr && k < a.m) {
        const int row = row0 + i, pos = pos_of[i], slot = slot_of[i];
        float current;
        u = conv_at<T>(a, row, STEP ? 0 : row - a.cu_rows[a.row_seq[row]], pos, slot, c0 + k, current);
        if (STEP && k >= o0 && k < o0 + 16) a.ring[(size_t(slot) * a.taps + pos % a.taps) * a.width + c0 + k] = current;
      }
      us[idx] = u;
    }
  }
  __syncthreads();
  float zr[kRows], zi[kRows];
#pragma unroll
  for (int i = 0; i < kRows; ++i) zr[i] = zi[i] = 0.0f;
  for (int k = 8 * lane16; k < a.m; k += 128) {
    float r8[8], i8[8];
    if (vec) {
      if (k >= 128) {
        raw8(raw_r, wr + k);
        raw8(raw_i, wi + k);
      }
      unpack8(raw_r, r8);
      unpack8(raw_i, i8);
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        r8[e] = k + e < a.m ? ld_f(wr, k + e) : 0.0f;
        i8[e] = k + e < a.m ? ld_f(wi, k + e) : 0.0f;
      }
    }
#pragma unroll
    for (int i = 0; i < kRows; ++i) {
      float u8[8];
      load8(us + i * padded + k, u8);
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        zr[i] = fmaf(r8[e], u8[e], zr[i]);
        zi[i] = fmaf(i8[e], u8[e], zi[i]);
      }
    }
  }
  // sums over the sixteen lanes: at every step a lane hands half of its numbers over and keeps the sums of the other half,
  // until lane l has row l % 8 of one of the two products (lanes 0 .. 7 the first)
  static_assert(kRows == 8, "sixteen lanes share the sums of eight rows of two products");
  float z[2 * kRows];
#pragma unroll
  for (int i = 0; i < kRows; ++i) { z[i] = zr[i]; z[kRows + i] = zi[i]; }
#pragma unroll
  for (int off = 8; off > 0; off >>= 1)
#pragma unroll
    for (int i = 0; i < off; ++i) {
      const bool up = lane16 & off;
      z[i] = (up ? z[off + i] : z[i]) + __shfl_xor(up ? z[i] : z[off + i], off, 64);
    }
  const float g = __shfl_xor(z[0], 8, 64);           // (of lanes 0 .. 7)
  if (!live || lane16 >= nr) return;
  const float2 ab = decay_and_input(z[0] + br, g + bi, us[lane16 * padded + o], rate);
  if (STEP) {
    S = fmaf(ab.x, S, ab.y);
    a.state[size_t(my_slot) * a.width + c] = S;
    float y;
    if (SL > 0) {
      y = y_in[0];
#pragma unroll
      for (int s = 1; s < SL; ++s)
        if (s < a.n_slices) y += y_in[s];
    } else {
      y = sum_slices(a.y + size_t(my_row) * a.row_stride + c, a.n_slices, a.slice_stride);
    }
    store_out(a, my_row, c, S, y + a.y_bias[c]);
  } else {
    a.ab[size_t(my_row) * a.width + c] = ab;
  }
}

// The inputs of a sequence's last positions go to their rows of the ring.
__device__ __forceinline__ void keep_inputs(const LruArgs &a, int r0, int r1, int slot, int c) {
  for (int row = max(r0, r1 - a.taps); row < r1; ++row)
    a.ring[(size_t(slot) * a.taps + a.row_pos[row] % a.taps) * a.width + c] = input_at(a, row, c);
}

__global__ void __launch_bounds__(256) lru_walk_kernel(LruArgs a) {
  const int seq = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
  if (c >= a.width) return;
  const int r0 = a.cu_rows[seq], r1 = a.cu_rows[seq + 1], slot = a.slots[seq];
  if (r1 <= r0) return;
  float S = a.state[size_t(slot) * a.width + c];
  for (int row = r0; row < r1; ++row) {
    const float2 ab = a.ab[size_t(row) * a.width + c];
    S = fmaf(ab.x, S, ab.y);
    store_out(a, row, c, S, sum_slices(a.y + size_t(row) * a.row_stride + c, a.n_slices, a.slice_stride) + a.y_bias[c]);
  }
  a.state[size_t(slot) * a.width + c] = S;
  keep_inputs(a, r0, r1, slot, c);
}

// (a, b) after (a', b'): S -> a (a' S + b') + b.
__device__ __forceinline__ float2 after(float2 later, float2 earlier) {
  return make_float2(later.x * earlier.x, fmaf(later.x, earlier.y, later.y));
}

// grid (chunks, blocks of channels).  The three parts of u lie in LDS, rows of `stride` bfloat16 numbers; a wave a
// sixteen of the block's channels.
template <int T>
__global__ void __launch_bounds__(512) lru_chunk_gates_kernel(LruArgs a) {
  extern __shared__ __attribute__((aligned(16))) bf16_t planes[];
  const int m32 = (a.m + 31) & ~31, stride = m32 + 8, plane = kChunk * stride;
  const int32_t *ch = a.chunks + 4 * size_t(blockIdx.x);
  const int r0 = ch[0], nr = ch[1], seq = ch[2];
  const int c0 = blockIdx.y * a.m, tid = threadIdx.x, threads = blockDim.x, lane = tid & 63, col = lane & 15, g = lane >> 4;
  const bf16_t *wr = (const bf16_t *)a.ra, *wi = (const bf16_t *)a.ri;
  const int n_ot = (a.m + 15) / 16, first_ot = min(tid >> 6, n_ot - 1);
  // what the wave's first sixteen channels need is asked for first
  constexpr int AHEAD = 4;               // steps of 32 of the products
  uint4 ahead[AHEAD][2];
  {
    const int o = 16 * first_ot + col, c = c0 + min(o, a.m - 1);
#pragma unroll
    for (int s = 0; s < AHEAD; ++s) {
      const int k = 32 * s + 8 * g;
      ahead[s][0] = ld16(wr + size_t(c) * a.m + k, k < a.m && o < a.m);
      ahead[s][1] = ld16(wi + size_t(c) * a.m + k, k < a.m && o < a.m);
    }
  }
  const int first = a.cu_rows[seq], slot = a.slots[seq], p0 = a.row_pos[r0];
  // a thread a channel and a part of sixteen rows: every input is read once and stays for the taps after it
  for (int item = tid; item < (kChunk / kPart) * m32; item += threads) {
    const int k = item % m32, part = item / m32, i0 = part * kPart;
    bf16_t *dst = planes + i0 * stride + k;
    float u[kPart];
    if (k >= a.m || i0 >= nr) {
#pragma unroll
      for (int i = 0; i < kPart; ++i) u[i] = 0.0f;
    } else if (T > 0) {
      constexpr int N = kPart + (T > 0 ? T : 1) - 1;
      float in[N];
#pragma unroll
      for (int j = 0; j < N; ++j) {
        // input i0 - (T - 1) + j of the chunk; rows past the chunk's last read the last again
        const int i = i0 - (T - 1) + j, row = r0 + min(i, nr - 1);
        in[j] = a.x[size_t(max(row, first)) * a.row_stride + c0 + k];
      }
      for (int s = 1; s < a.n_slices; ++s)
#pragma unroll
        for (int j = 0; j < N; ++j)
          in[j] += a.x[s * a.slice_stride + size_t(max(r0 + min(i0 - (T - 1) + j, nr - 1), first)) * a.row_stride + c0 + k];
      const float bx = a.x_bias[c0 + k];
#pragma unroll
      for (int j = 0; j < N; ++j) in[j] += bx;
      if (r0 + i0 - (T - 1) < first) {      // the sequence's first part of the step: inputs of earlier steps
#pragma unroll
        for (int j = 0; j < T - 1; ++j) {
          const int i = i0 - (T - 1) + j, p = p0 + i;
          if (r0 + i < first) in[j] = p >= 0 ? a.ring[(size_t(slot) * T + p % (T > 0 ? T : 1)) * a.width + c0 + k] : 0.0f;
        }
      }
      float w[T > 0 ? T : 1];
#pragma unroll
      for (int j = 0; j < T; ++j) w[j] = a.taps_w[size_t(c0 + k) * T + j];
      const float b = a.taps_b[c0 + k];
#pragma unroll
      for (int i = 0; i < kPart; ++i) {
        float acc = 0.0f;
#pragma unroll
        for (int j = 0; j < T; ++j) acc = fmaf(w[j], in[i + j], acc);
        u[i] = i0 + i < nr ? acc + b : 0.0f;
      }
    } else {
      for (int i = 0; i < kPart; ++i) {
        float current;
        u[i] = 0.0f;
        if (i0 + i < nr) u[i] = conv_at<0>(a, r0 + i0 + i, r0 + i0 + i - first, p0 + i0 + i, slot, c0 + k, current);
      }
    }
#pragma unroll
    for (int i = 0; i < kPart; i += 2) {         // two rows a conversion
      float f0 = u[i], f1 = u[i + 1];
#pragma unroll
      for (int p = 0; p < 3; ++p) {
        const uint32_t w = pack_bf16(f0, f1);
        dst[p * plane + i * stride] = bf16_t(w & 0xffffu);
        dst[p * plane + (i + 1) * stride] = bf16_t(w >> 16);
        f0 -= __uint_as_float(w << 16);
        f1 -= __uint_as_float(w & 0xffff0000u);
      }
    }
  }
  __syncthreads();
  for (int ot = tid >> 6; ot < n_ot; ot += threads >> 6) {
    const int o = 16 * ot + col, c = c0 + min(o, a.m - 1);
    floatx4_t zr[kChunk / 16], zi[kChunk / 16];
#pragma unroll
    for (int t = 0; t < kChunk / 16; ++t) zr[t] = zi[t] = floatx4_t{0.f, 0.f, 0.f, 0.f};
    auto product = [&](int k, uint4 w0, uint4 w1) {
      const bf16x8_t fr = as_bf16x8(w0), fi = as_bf16x8(w1);
#pragma unroll
      for (int p = 2; p >= 0; --p)
#pragma unroll
        for (int t = 0; t < kChunk / 16; ++t) {
          const bf16x8_t fu = as_bf16x8(*reinterpret_cast<const uint4 *>(planes + p * plane + (16 * t + col) * stride + k));
          zr[t] = mfma16(fu, fr, zr[t]);
          zi[t] = mfma16(fu, fi, zi[t]);
        }
    };
    const float br = a.ra_b[c], bi = a.ri_b[c], rate = a.rate[c];
    int s0 = 0;
    if (ot == first_ot) {
#pragma unroll
      for (int s = 0; s < AHEAD; ++s)
        if (32 * s < m32) product(32 * s + 8 * g, ahead[s][0], ahead[s][1]);
      s0 = AHEAD;
    }
    for (int k = 32 * s0 + 8 * g; k < m32; k += 32) {
      const bool in = k < a.m && o < a.m;
      product(k, ld16(wr + size_t(c) * a.m + k, in), ld16(wi + size_t(c) * a.m + k, in));
    }
    // a lane has rows 16 t + 4 g .. + 3 of channel o
    float2 total = make_float2(1.0f, 0.0f);
#pragma unroll
    for (int t = 0; t < kChunk / 16; ++t) {
      float2 f = make_float2(1.0f, 0.0f);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int i = 16 * t + 4 * g + e;
        const bf16_t *at = planes + i * stride + min(o, a.m - 1);
        const float u = (bf16_to_f32(at[2 * plane]) + bf16_to_f32(at[plane])) + bf16_to_f32(at[0]);
        const float2 ab = decay_and_input(zr[t][e] + br, zi[t][e] + bi, u, rate);
        if (i < nr) {
          f = after(ab, f);
          if (o < a.m) a.ab[size_t(r0 + i) * a.width + c] = ab;
        }
      }
      // over the four lanes of the channel, in the order of their rows
      float2 n = make_float2(__shfl_xor(f.x, 16, 64), __shfl_xor(f.y, 16, 64));
      f = (g & 1) ? after(f, n) : after(n, f);
      n = make_float2(__shfl_xor(f.x, 32, 64), __shfl_xor(f.y, 32, 64));
      f = (g & 2) ? after(f, n) : after(n, f);
      total = after(f, total);
    }
    if (g == 0 && o < a.m) a.folded[size_t(blockIdx.x) * a.width + c] = total;
  }
}

// The state at the start of every chunk in place of its folded pair's first number; the state after a sequence's last
// chunk goes to state[], its last inputs to the ring.
__global__ void __launch_bounds__(64) lru_carry_kernel(LruArgs a) {
  constexpr int AHEAD = 16;
  const int seq = blockIdx.y, c = blockIdx.x * 64 + threadIdx.x;
  if (c >= a.width) return;
  const int r0 = a.cu_rows[seq], r1 = a.cu_rows[seq + 1], slot = a.slots[seq];
  if (r1 <= r0) return;
  int lo = 0, hi = a.n_chunks;        // the chunks lie in the order of the rows: the sequence's are together
  while (lo < hi) {
    const int mid = (lo + hi) >> 1;
    if (a.chunks[4 * mid + 2] < seq) lo = mid + 1;
    else hi = mid;
  }
  const int n = (r1 - r0 + kChunk - 1) / kChunk;
  float S = a.state[size_t(slot) * a.width + c];
  float2 *p = a.folded + size_t(lo) * a.width + c;
  for (int i = 0; i < n; i += AHEAD) {
    float2 f[AHEAD];
#pragma unroll
    for (int j = 0; j < AHEAD; ++j) f[j] = p[size_t(min(i + j, n - 1)) * a.width];
#pragma unroll
    for (int j = 0; j < AHEAD; ++j)
      if (i + j < n) {
        p[size_t(i + j) * a.width].x = S;
        S = fmaf(f[j].x, S, f[j].y);
      }
  }
  a.state[size_t(slot) * a.width + c] = S;
  keep_inputs(a, r0, r1, slot, c);
}

// A block 64 channels of a chunk; a wave a part of sixteen rows, all of whose pairs it asks for at once.
__global__ void __launch_bounds__(256) lru_chunk_walk_kernel(LruArgs a) {
  __shared__ float2 folds[kChunk / kPart][64];
  const int32_t *ch = a.chunks + 4 * size_t(blockIdx.y);
  const int r0 = ch[0], nr = ch[1], lane = threadIdx.x & 63, part = threadIdx.x >> 6, i0 = part * kPart;
  const int c = min(int(blockIdx.x) * 64 + lane, a.width - 1);
  float2 ab[kPart];
  float y[kPart];
#pragma unroll
  for (int i = 0; i < kPart; ++i) {
    const int row = r0 + min(i0 + i, nr - 1);
    ab[i] = a.ab[size_t(row) * a.width + c];
    y[i] = a.y[size_t(row) * a.row_stride + c];
  }
  for (int s = 1; s < a.n_slices; ++s)
#pragma unroll
    for (int i = 0; i < kPart; ++i) y[i] += a.y[s * a.slice_stride + size_t(r0 + min(i0 + i, nr - 1)) * a.row_stride + c];
  float S = a.folded[size_t(blockIdx.y) * a.width + c].x;
  const float by = a.y_bias[c];
  float2 f = make_float2(1.0f, 0.0f);
#pragma unroll
  for (int i = 0; i < kPart; ++i)
    if (i0 + i < nr) f = after(ab[i], f);
  folds[part][lane] = f;
  __syncthreads();
  for (int p = 0; p < part; ++p) S = fmaf(folds[p][lane].x, S, folds[p][lane].y);
  if (int(blockIdx.x) * 64 + lane >= a.width) return;
#pragma unroll
  for (int i = 0; i < kPart; ++i)
    if (i0 + i < nr) {
      S = fmaf(ab[i].x, S, ab[i].y);
      store_out(a, r0 + i0 + i, c, S, y[i] + by);
    }
}

template <typename TW, int SL>
void launch_step(const LruArgs &a, dim3 grid, size_t lds, int vec, hipStream_t s) {
  if (a.taps == 2) lru_gates_kernel<TW, 2, true, SL><<<grid, 256, lds, s>>>(a, vec);
  else if (a.taps == 3) lru_gates_kernel<TW, 3, true, SL><<<grid, 256, lds, s>>>(a, vec);
  else if (a.taps == 4) lru_gates_kernel<TW, 4, true, SL><<<grid, 256, lds, s>>>(a, vec);
  else lru_gates_kernel<TW, 0, true, SL><<<grid, 256, lds, s>>>(a, vec);
}

template <typename TW, bool STEP>
void launch_gates(const LruArgs &a, hipStream_t s) {
  const dim3 grid((a.width / a.m) * ((a.m + 15) / 16), (a.n_rows + kRows - 1) / kRows);
  const size_t lds = size_t(kRows) * ((a.m + 7) & ~7) * sizeof(float);
  const int vec = a.m % 8 == 0 && (reinterpret_cast<uintptr_t>(a.ra) & 15) == 0 && (reinterpret_cast<uintptr_t>(a.ri) & 15) == 0;
  if constexpr (STEP) {
    if (a.n_slices == 1) launch_step<TW, 1>(a, grid, lds, vec, s);
    else if (a.n_slices <= 8) launch_step<TW, 8>(a, grid, lds, vec, s);
    else lru_gates_kernel<TW, 0, true, 0><<<grid, 256, lds, s>>>(a, vec);
  } else {
    lru_gates_kernel<TW, 0, false, 0><<<grid, 256, lds, s>>>(a, vec);
  }
}

template <int T>
int launch_chunk_gates(const LruArgs &a, hipStream_t s) {
  const size_t lds = size_t(3) * kChunk * (((a.m + 31) & ~31) + 8) * sizeof(bf16_t);
  if (lds > 65536) {
    if (hipFuncSetAttribute((const void *)lru_chunk_gates_kernel<T>, hipFuncAttributeMaxDynamicSharedMemorySize, int(lds)) != hipSuccess) {
      (void)hipGetLastError();
      return sb::fail(SB_ERR_UNSUPPORTED, "sb_gated_lru: blocks of %d channels do not fit LDS", a.m);
    }
  }
  const int waves = min(8, (a.m + 15) / 16);
  lru_chunk_gates_kernel<T><<<dim3(a.n_chunks, a.width / a.m), 64 * waves, lds, s>>>(a);
  return SB_OK;
}

}  // namespace

extern "C" int sb_gated_lru_max_taps(void) { return kMaxTaps; }
extern "C" int sb_gated_lru_max_block(void) { return kMaxBlock; }
extern "C" int sb_gated_lru_chunk_rows(void) { return kChunk; }
// whether the chunked form takes blocks of m channels with weights of this type
extern "C" int sb_gated_lru_chunked_ok(int m, int w_dtype) { return w_dtype == SB_BF16 && m % 8 == 0 && m <= kMaxBlockMfma; }

// x, y: float32 columns of the same rows (row_stride numbers apart, whole or in K slices); ab f32 [rows, width, 2] scratch
// (NULL when every sequence brings one row); chunks int32 [n_chunks, 4] with folded f32 [n_chunks, width, 2] scratch for the
// chunked form, or NULL.
extern "C" int sb_gated_lru(void *out, int out_dtype, const float *x, const float *y, int row_stride, int n_slices, size_t slice_stride,
                            const float *x_bias, const float *y_bias, const float *taps_w, const float *taps_b, int taps, const void *ra,
                            const void *ri, int w_dtype, const float *ra_b, const float *ri_b, const float *rate, float *state,
                            float *ring, const int32_t *row_pos, const int32_t *row_seq, const int32_t *cu_rows, const int32_t *slots,
                            int n_rows, int n_seqs, int width, int block, float *ab, const int32_t *chunks, int n_chunks, float *folded,
                            void *stream) {
  SB_REQUIRE(out && x && y && x_bias && y_bias && taps_w && taps_b && ra && ri && ra_b && ri_b && rate && state && ring && row_pos &&
                 row_seq && cu_rows && slots, "sb_gated_lru: null pointer");
  SB_REQUIRE(n_rows >= 0 && n_seqs >= 0 && n_slices > 0 && width > 0 && block > 0 && width % block == 0 && taps > 0 && row_stride >= width,
             "sb_gated_lru: bad sizes rows=%d width=%d block=%d taps=%d", n_rows, width, block, taps);
  SB_REQUIRE(sb::valid_dtype(out_dtype) && sb::valid_dtype(w_dtype), "sb_gated_lru: unknown dtype");
  SB_SUPPORT(taps <= kMaxTaps && block <= kMaxBlock, "sb_gated_lru: %d taps and blocks of %d are more than %d and %d", taps, block,
             kMaxTaps, kMaxBlock);
  SB_SUPPORT(n_seqs <= 65535 && n_rows <= 65535 * kRows && width / block <= 65535 && n_chunks <= 65535,
             "sb_gated_lru: too many rows, sequences, chunks or blocks");
  if (n_rows == 0 || n_seqs == 0) return SB_OK;
  const LruArgs a{out, out_dtype, x, y, row_stride, n_slices, slice_stride, x_bias, y_bias, taps_w, taps_b, taps, ra, ri, w_dtype, ra_b,
                  ri_b, rate, state, ring, row_pos, row_seq, cu_rows, slots, n_rows, n_seqs, width, block, (float2 *)ab, chunks, n_chunks,
                  (float2 *)folded};
  hipStream_t s = (hipStream_t)stream;
  if (n_rows == n_seqs && !chunks) {
    if (w_dtype == SB_F32) launch_gates<float, true>(a, s);
    else launch_gates<bf16_t, true>(a, s);
    return sb::check_launch("sb_gated_lru");
  }
  SB_REQUIRE(ab && (reinterpret_cast<uintptr_t>(ab) & 7) == 0, "sb_gated_lru: several rows a sequence need their scratch");
  if (!chunks) {
    if (w_dtype == SB_F32) launch_gates<float, false>(a, s);
    else launch_gates<bf16_t, false>(a, s);
    lru_walk_kernel<<<dim3((width + 255) / 256, n_seqs), 256, 0, s>>>(a);
    return sb::check_launch("sb_gated_lru");
  }
  SB_REQUIRE(n_chunks > 0 && folded && (reinterpret_cast<uintptr_t>(folded) & 7) == 0, "sb_gated_lru: the chunked form needs its scratch");
  SB_SUPPORT(sb_gated_lru_chunked_ok(block, w_dtype) && (reinterpret_cast<uintptr_t>(ra) & 15) == 0 && (reinterpret_cast<uintptr_t>(ri) & 15) == 0,
             "sb_gated_lru: the chunked form takes bfloat16 weights and blocks of up to %d channels in eights", kMaxBlockMfma);
  int e;
  if (taps == 2) e = launch_chunk_gates<2>(a, s);
  else if (taps == 3) e = launch_chunk_gates<3>(a, s);
  else if (taps == 4) e = launch_chunk_gates<4>(a, s);
  else e = launch_chunk_gates<0>(a, s);
  if (e != SB_OK) return e;
  lru_carry_kernel<<<dim3((width + 63) / 64, n_seqs), 64, 0, s>>>(a);
  lru_chunk_walk_kernel<<<dim3((width + 63) / 64, n_chunks), 256, 0, s>>>(a);
  return sb::check_launch("sb_gated_lru");
}
