// The pass that ends a block whose branches read one normed stream, and the layer norm.
//
//   out[r,:] = base[r,:] + sum_b scale_b N_b(sum_s part_b[s][r,:]) + vec
//   N_b: the sum as it is, or divided by its root mean square (eps inside the root) times a weight;
//   h[r,:]: what the next block reads, from the same pass: out's RMS norm or layer norm
//   ((x - mean) / sqrt(mean((x - mean)^2) + eps) * w), or out itself in the activation type.
// Without branches, `out` and `vec` it is a norm of its own (sb_layernorm), of rows picked by `rows`.
//
// Sums over a row in double, per thread in ascending order, a fixed butterfly over the wave, the waves in
// ascending order: with one block shape a row's bits depend on the row alone.  Rows in fours that fit the
// block's registers: a thread keeps its groups of four and asks for every slice of every branch before it
// adds any.  Other widths go through LDS.
#include "common.h"

namespace {

constexpr int kMaxTerms = 3;
constexpr int kMaxSlices = 24;         // of all branches together
enum { THEN_NOTHING = 0, THEN_RMS = 1, THEN_LAYER = 2, THEN_COPY = 3 };

struct Term {
  const float *part; int n_slices; size_t slice_stride;
  const void *w; int w_dtype; int norm; float scale;
};
struct JoinArgs {
  float *out; const float *base; const int32_t *rows;
  Term t[kMaxTerms]; float term_eps;
  const void *vec; int vec_dtype;
  void *h; int h_dtype, then; const void *hw; int hw_dtype; float h_eps;
  int width;
  // the branches' slices one after the other (places past the last hold the last again), and where each branch ends
  const float *slice[kMaxSlices]; int end[kMaxTerms];
};

template <int THREADS, int N>
__device__ __forceinline__ void block_sums(double (&v)[N], double (*slots)[N]) {
#pragma unroll
  for (int n = 0; n < N; ++n) v[n] = wave_sum(v[n]);
  if ((threadIdx.x & 63) == 0)
#pragma unroll
    for (int n = 0; n < N; ++n) slots[threadIdx.x >> 6][n] = v[n];
  __syncthreads();
#pragma unroll
  for (int n = 0; n < N; ++n) {
    double s = 0.0;
#pragma unroll
    for (int k = 0; k < THREADS / 64; ++k) s += slots[k][n];
    v[n] = s;
  }
}

__device__ __forceinline__ float inv_root(double mean_sq, float eps) { return 1.0f / sqrtf(float(mean_sq) + eps); }

// mean and 1 / deviation of a row from its sum and its sum of squares (both in double)
__device__ __forceinline__ void row_norm(const double (&s)[2], int width, int then, float eps, float &mean, float &inv) {
  const double m = then == THEN_LAYER ? s[0] / double(width) : 0.0;
  const double var = s[1] / double(width) - m * m;
  mean = float(m);
  inv = inv_root(var > 0.0 ? var : 0.0, eps);
}

template <int NT, int THREADS, int KEEP, int SL>      // SL: slices the unrolled loops ask for (>= those of all branches)
__global__ void __launch_bounds__(THREADS) join_kernel(JoinArgs a) {
  __shared__ double term_slots[THREADS / 64][NT > 0 ? NT : 1], row_slots[THREADS / 64][2];
  const int r = blockIdx.x, tid = threadIdx.x, n_groups = a.width / 4;
  const size_t from = size_t(a.rows ? a.rows[r] : r) * n_groups, at = size_t(r) * n_groups;
  float4 in[KEEP][NT > 0 ? SL : 1], base[KEEP];
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int g = min(tid + i * THREADS, n_groups - 1);
    if (NT > 0)
#pragma unroll
      for (int s = 0; s < SL; ++s) in[i][s] = reinterpret_cast<const float4 *>(a.slice[s])[at + g];
    base[i] = reinterpret_cast<const float4 *>(a.base)[from + g];
  }
  float4 y[NT > 0 ? NT : 1][KEEP];
  double sq[NT > 0 ? NT : 1];
  bool any_norm = false;
#pragma unroll
  for (int b = 0; b < NT; ++b)
#pragma unroll
    for (int i = 0; i < KEEP; ++i) y[b][i] = make_float4(0.f, 0.f, 0.f, 0.f);
  if (NT > 0) {
#pragma unroll
    for (int s = 0; s < SL; ++s)
#pragma unroll
      for (int b = 0; b < NT; ++b)
        if (s < a.end[b] && (b == 0 || s >= a.end[b > 0 ? b - 1 : 0])) {      // (the same for all lanes)
#pragma unroll
          for (int i = 0; i < KEEP; ++i) { y[b][i].x += in[i][s].x; y[b][i].y += in[i][s].y; y[b][i].z += in[i][s].z; y[b][i].w += in[i][s].w; }
        }
  }
#pragma unroll
  for (int b = 0; b < NT; ++b) {
    sq[b] = 0.0;
    any_norm = any_norm || a.t[b].norm;
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
      const float4 v = y[b][i];
      if (tid + i * THREADS < n_groups)
        sq[b] += double(v.x * v.x) + double(v.y * v.y) + double(v.z * v.z) + double(v.w * v.w);
    }
  }
  if (NT > 0 && any_norm) block_sums<THREADS>(sq, term_slots);
  float4 x[KEEP];
  double s2[2] = {0.0, 0.0};
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int g = min(tid + i * THREADS, n_groups - 1);
    float add[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int b = 0; b < NT; ++b) {
      const float v[4] = {y[b][i].x, y[b][i].y, y[b][i].z, y[b][i].w};
      const float inv = a.t[b].norm ? inv_root(sq[b] / double(a.width), a.term_eps) : 1.0f;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        float z = v[e];
        if (a.t[b].norm) z = a.t[b].w ? (z * inv) * ld_dyn(a.t[b].w, a.t[b].w_dtype, 4 * g + e) : z * inv;
        add[e] += a.t[b].scale == 1.0f ? z : a.t[b].scale * z;
      }
    }
    float4 v = base[i];
    if (NT > 0) { v.x += add[0]; v.y += add[1]; v.z += add[2]; v.w += add[3]; }
    if (a.vec) {
      v.x += ld_dyn(a.vec, a.vec_dtype, 4 * g); v.y += ld_dyn(a.vec, a.vec_dtype, 4 * g + 1);
      v.z += ld_dyn(a.vec, a.vec_dtype, 4 * g + 2); v.w += ld_dyn(a.vec, a.vec_dtype, 4 * g + 3);
    }
    x[i] = v;
    if (tid + i * THREADS < n_groups) {
      if (a.out) reinterpret_cast<float4 *>(a.out)[at + g] = v;
      s2[0] += (double(v.x) + double(v.y)) + (double(v.z) + double(v.w));
      s2[1] += (double(v.x) * double(v.x) + double(v.y) * double(v.y)) + (double(v.z) * double(v.z) + double(v.w) * double(v.w));
    }
  }
  if (a.then == THEN_NOTHING) return;
  float mean = 0.0f, inv = 1.0f;
  if (a.then != THEN_COPY) {
    block_sums<THREADS>(s2, row_slots);
    row_norm(s2, a.width, a.then, a.h_eps, mean, inv);
  }
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int g = tid + i * THREADS;
    if (g >= n_groups) continue;
    float o[4] = {x[i].x, x[i].y, x[i].z, x[i].w};
    if (a.then != THEN_COPY)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        o[e] = (o[e] - mean) * inv;
        if (a.hw) o[e] *= ld_dyn(a.hw, a.hw_dtype, 4 * g + e);
      }
    if (a.h_dtype == SB_BF16) {
      uint2 w2;
      w2.x = uint32_t(f32_to_bf16(o[0])) | uint32_t(f32_to_bf16(o[1])) << 16;
      w2.y = uint32_t(f32_to_bf16(o[2])) | uint32_t(f32_to_bf16(o[3])) << 16;
      reinterpret_cast<uint2 *>(a.h)[at + g] = w2;
    } else {
      reinterpret_cast<float4 *>(a.h)[at + g] = make_float4(o[0], o[1], o[2], o[3]);
    }
  }
}

// any width: the row and a branch's sum lie in LDS
__global__ void __launch_bounds__(256) join_any_kernel(JoinArgs a, int n_terms) {
  extern __shared__ float lds[];
  __shared__ double term_slots[4][1], row_slots[4][2];
  float *add = lds, *y = lds + a.width;
  const int r = blockIdx.x, tid = threadIdx.x;
  const size_t from = size_t(a.rows ? a.rows[r] : r) * a.width, at = size_t(r) * a.width;
  for (int i = tid; i < a.width; i += 256) add[i] = 0.0f;
  for (int b = 0; b < n_terms; ++b) {
    const Term &t = a.t[b];
    double sq[1] = {0.0};
    for (int i = tid; i < a.width; i += 256) {
      float v = t.part[at + i];
      for (int s = 1; s < t.n_slices; ++s) v += t.part[s * t.slice_stride + at + i];
      y[i] = v;
      sq[0] += double(v * v);
    }
    float inv = 1.0f;
    if (t.norm) {
      __syncthreads();        // the sums before this one have been read
      block_sums<256>(sq, term_slots);
      inv = inv_root(sq[0] / double(a.width), a.term_eps);
    }
    for (int i = tid; i < a.width; i += 256) {
      float z = y[i];
      if (t.norm) z = t.w ? (z * inv) * ld_dyn(t.w, t.w_dtype, i) : z * inv;
      add[i] += t.scale == 1.0f ? z : t.scale * z;
    }
  }
  double s2[2] = {0.0, 0.0};
  for (int i = tid; i < a.width; i += 256) {
    float v = a.base[from + i];
    if (n_terms > 0) v += add[i];
    if (a.vec) v += ld_dyn(a.vec, a.vec_dtype, i);
    add[i] = v;
    if (a.out) a.out[at + i] = v;
    s2[0] += double(v);
    s2[1] += double(v) * double(v);
  }
  if (a.then == THEN_NOTHING) return;
  float mean = 0.0f, inv = 1.0f;
  if (a.then != THEN_COPY) {
    block_sums<256>(s2, row_slots);
    row_norm(s2, a.width, a.then, a.h_eps, mean, inv);
  }
  for (int i = tid; i < a.width; i += 256) {
    float o = add[i];
    if (a.then != THEN_COPY) {
      o = (o - mean) * inv;
      if (a.hw) o *= ld_dyn(a.hw, a.hw_dtype, i);
    }
    if (a.h_dtype == SB_BF16) ((bf16_t *)a.h)[at + i] = f32_to_bf16(o);
    else ((float *)a.h)[at + i] = o;
  }
}

// the branches' loads of a thread that its registers hold (four numbers each): the rest goes through LDS
template <int NT, int THREADS, int KEEP, int SL>
bool launch_keep(const JoinArgs &a, int n_rows, hipStream_t s) {
  if constexpr (KEEP * SL > (THREADS > 256 ? (KEEP == 1 ? 24 : 14) : 48)) return false;
  else join_kernel<NT, THREADS, KEEP, SL><<<n_rows, THREADS, 0, s>>>(a);
  return true;
}

template <int NT, int THREADS, int SL>
bool launch_sl(const JoinArgs &a, int n_rows, hipStream_t s) {
  const int need = (a.width / 4 + THREADS - 1) / THREADS;
  if (need <= 1) return launch_keep<NT, THREADS, 1, SL>(a, n_rows, s);
  if (need <= 2) return launch_keep<NT, THREADS, 2, SL>(a, n_rows, s);
  if (need <= 4) return launch_keep<NT, THREADS, 4, SL>(a, n_rows, s);
  return false;
}

template <int NT, int THREADS>
bool launch_threads(const JoinArgs &a, int slices, int n_rows, hipStream_t s) {
  if constexpr (NT == 0) return launch_sl<NT, THREADS, 1>(a, n_rows, s);
  if (slices <= NT) return launch_sl<NT, THREADS, NT == 0 ? 1 : NT>(a, n_rows, s);
  if (slices <= 6) return launch_sl<NT, THREADS, 6>(a, n_rows, s);
  if (slices <= 12) return launch_sl<NT, THREADS, 12>(a, n_rows, s);
  if (slices <= 18) return launch_sl<NT, THREADS, 18>(a, n_rows, s);
  return launch_sl<NT, THREADS, 24>(a, n_rows, s);
}

template <int NT>
bool launch_fast(const JoinArgs &a, int slices, int n_rows, bool few, hipStream_t s) {
  if (few && a.width <= 2048 && launch_threads<NT, 512>(a, slices, n_rows, s)) return true;
  if ((few || a.width > 4096) && launch_threads<NT, 1024>(a, slices, n_rows, s)) return true;
  return a.width <= 4096 && launch_threads<NT, 256>(a, slices, n_rows, s);       // (wide rows: one shape for all row counts)
}

int launch_join(JoinArgs &a, int n_terms, int n_rows, int few, hipStream_t s, const char *what) {
  int slices = 0;
  bool ok = a.width % 4 == 0;
  const auto aligned = [](const void *p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  ok = ok && aligned(a.base) && aligned(a.out) && aligned(a.h);
  for (int b = 0; b < n_terms; ++b) {
    for (int i = 0; i < a.t[b].n_slices; ++i, ++slices)
      if (slices < kMaxSlices) a.slice[slices] = a.t[b].part + size_t(i) * a.t[b].slice_stride;
    a.end[b] = slices;
    ok = ok && aligned(a.t[b].part) && a.t[b].slice_stride % 4 == 0;
  }
  if (ok && slices <= kMaxSlices) {
    if (slices > 0)
      for (int i = slices; i < kMaxSlices; ++i) a.slice[i] = a.slice[slices - 1];
    bool done = false;
    const bool f = few && n_rows <= 64;
    if (n_terms == 0) done = launch_fast<0>(a, 1, n_rows, f, s);
    else if (n_terms == 1) done = launch_fast<1>(a, slices, n_rows, f, s);
    else if (n_terms == 2) done = launch_fast<2>(a, slices, n_rows, f, s);
    else done = launch_fast<3>(a, slices, n_rows, f, s);
    if (done) return sb::check_launch(what);
  }
  SB_SUPPORT(a.width <= 8192, "%s: rows of %d with these branches are wider than 8192", what, a.width);
  join_any_kernel<<<n_rows, 256, size_t(2) * a.width * sizeof(float), s>>>(a, n_terms);
  return sb::check_launch(what);
}

}  // namespace

// n_terms <= 3; term_ptrs: per branch {part, weight or NULL}; term_ints: per branch {slices, weight dtype, norm};
// slice strides in numbers; base may be out.  few: wider blocks for up to 64 rows (the order of a row's sums
// then depends on the number of rows).
extern "C" int sb_join(float *out, const float *base, const void *const *term_ptrs, const int *term_ints,
                       const float *term_scales, const size_t *slice_strides, int n_terms, float term_eps, const void *vec,
                       int vec_dtype, void *h, int h_dtype, int then, const void *h_weight, int h_w_dtype, float h_eps,
                       int n_rows, int width, int few, void *stream) {
  SB_REQUIRE(out && base && (n_terms == 0 || (term_ptrs && term_ints && term_scales && slice_strides)), "sb_join: null pointer");
  SB_REQUIRE(n_rows >= 0 && width > 0 && n_terms >= 0, "sb_join: bad sizes rows=%d width=%d branches=%d", n_rows, width, n_terms);
  SB_SUPPORT(n_terms <= kMaxTerms, "sb_join: %d branches, at most %d", n_terms, kMaxTerms);
  SB_REQUIRE(then >= THEN_NOTHING && then <= THEN_COPY && (then == THEN_NOTHING || (h && sb::valid_dtype(h_dtype))) &&
                 (!h_weight || sb::valid_dtype(h_w_dtype)) && (!vec || sb::valid_dtype(vec_dtype)),
             "sb_join: bad norm or type after the sum");
  if (n_rows == 0) return SB_OK;
  JoinArgs a{};
  a.out = out; a.base = base; a.rows = nullptr; a.term_eps = term_eps; a.vec = vec; a.vec_dtype = vec_dtype;
  a.h = h; a.h_dtype = h_dtype; a.then = then; a.hw = h_weight; a.hw_dtype = h_w_dtype; a.h_eps = h_eps; a.width = width;
  for (int b = 0; b < n_terms; ++b) {
    a.t[b] = Term{(const float *)term_ptrs[2 * b], term_ints[3 * b], slice_strides[b], term_ptrs[2 * b + 1], term_ints[3 * b + 1],
                  term_ints[3 * b + 2], term_scales[b]};
    SB_REQUIRE(a.t[b].part && a.t[b].n_slices >= 1 && (!a.t[b].w || sb::valid_dtype(a.t[b].w_dtype)), "sb_join: bad branch %d", b);
  }
  return launch_join(a, n_terms, n_rows, few, (hipStream_t)stream, "sb_join");
}

// y[r,:] = (x - mean) / sqrt(mean((x - mean)^2) + eps) * w of row rows[r] (NULL: r); w may be NULL.
extern "C" int sb_layernorm(void *y, int out_dtype, const float *x, const void *w, int w_dtype, const int32_t *rows,
                            int n_rows, int width, float eps, int few, void *stream) {
  SB_REQUIRE(y && x, "sb_layernorm: null pointer");
  SB_REQUIRE(n_rows >= 0 && width > 0, "sb_layernorm: bad sizes rows=%d width=%d", n_rows, width);
  SB_REQUIRE(sb::valid_dtype(out_dtype) && (!w || sb::valid_dtype(w_dtype)), "sb_layernorm: unknown dtype");
  if (n_rows == 0) return SB_OK;
  JoinArgs a{};
  a.base = x; a.rows = rows; a.h = y; a.h_dtype = out_dtype; a.then = THEN_LAYER; a.hw = w; a.hw_dtype = w_dtype; a.h_eps = eps;
  a.width = width;
  return launch_join(a, 0, n_rows, few, (hipStream_t)stream, "sb_layernorm");
}
