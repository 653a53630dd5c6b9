// A residual kept as several streams that mix (hyper-connections): a row of the stream is S rows X_1 .. X_S of
// `width` float32 numbers side by side.
//
//   sb_streams_embed   X_1 = .. = X_S = table[id]
//   sb_streams_join    the pass that ends a sublayer and starts the next one:
//       y    = sum_i a_i(row) part_i[row,:] + vec        (a product's K slices, experts' results, branches)
//       X_t <- sum_s mix[s][t] X_s + out[t] y            (all t from the old streams)
//       h    = r(sum_t in[t] X_t) * w                    (r: divided by the root mean square, eps inside the root)
//   sb_streams_read    h alone, of picked rows (in NULL: the plain sum of the streams)
//
// Sums of squares in double, per thread in ascending order, a fixed butterfly over the wave, the waves in ascending
// order: with one block shape a row's bits depend on the row alone.  A thread keeps its columns of all streams in
// registers and asks for everything it reads before it adds any.
#include "common.h"

namespace {

constexpr int kMaxStreams = 16;
constexpr int kMaxSlices = 32;
constexpr int kMaxWidth = 16384;

struct StreamArgs {
  float *x; const int32_t *rows;
  // part i of the sublayer's result: row r lies at part[i] + r * part_stride[i], counts part_scale[i] times (times
  // part_w[i][r * part_w_stride[i]] when that is given)
  const float *part[kMaxSlices]; int part_stride[kMaxSlices]; float part_scale[kMaxSlices];
  const float *part_w[kMaxSlices]; int part_w_stride[kMaxSlices];
  int n_parts;
  const void *vec; int vec_dtype;
  const float *mix, *out, *in;
  void *h; int h_dtype; const void *w; int w_dtype; float eps;
  int streams, width, store;
};

template <int THREADS>
__device__ __forceinline__ double block_total(double v) {
  __shared__ double slots[THREADS / 64];
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) slots[threadIdx.x >> 6] = v;
  __syncthreads();
  double s = 0.0;
#pragma unroll
  for (int k = 0; k < THREADS / 64; ++k) s += slots[k];
  return s;
}

__device__ __forceinline__ float part_factor(const StreamArgs &a, int i, int r) {
  return a.part_w[i] ? a.part_scale[i] * a.part_w[i][size_t(r) * a.part_w_stride[i]] : a.part_scale[i];
}

__device__ __forceinline__ float4 fma4(float c, float4 v, float4 acc) {
  acc.x = fmaf(c, v.x, acc.x); acc.y = fmaf(c, v.y, acc.y); acc.z = fmaf(c, v.z, acc.z); acc.w = fmaf(c, v.w, acc.w);
  return acc;
}

// Rows in fours.  S streams, P: parts the unrolled loops ask for (>= n_parts; places past the last hold the last again
// and are not added), KEEP groups of four columns a thread.
template <int S, int P, int THREADS, int KEEP>
__global__ void __launch_bounds__(THREADS) streams_kernel(StreamArgs a) {
  const int r = blockIdx.x, tid = threadIdx.x, n_groups = a.width / 4;
  const size_t src = size_t(a.rows ? a.rows[r] : r) * S * n_groups;
  float4 *x4 = reinterpret_cast<float4 *>(a.x);
  float4 in[KEEP][P > 0 ? P : 1], x[KEEP][S];
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int g = min(tid + k * THREADS, n_groups - 1);
#pragma unroll
    for (int i = 0; i < P; ++i) in[k][i] = reinterpret_cast<const float4 *>(a.part[i] + size_t(r) * a.part_stride[i])[g];
#pragma unroll
    for (int s = 0; s < S; ++s) x[k][s] = x4[src + size_t(s) * n_groups + g];
  }
  if (a.store) {
    float c[P > 0 ? P : 1];
#pragma unroll
    for (int i = 0; i < P; ++i) c[i] = i < a.n_parts ? part_factor(a, i, r) : 0.0f;
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
      const int g = min(tid + k * THREADS, n_groups - 1);
      float4 y = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
      for (int i = 0; i < P; ++i)
        if (i < a.n_parts) y = fma4(c[i], in[k][i], y);      // (the same for all lanes)
      if (a.vec) {
        y.x += ld_dyn(a.vec, a.vec_dtype, 4 * g); y.y += ld_dyn(a.vec, a.vec_dtype, 4 * g + 1);
        y.z += ld_dyn(a.vec, a.vec_dtype, 4 * g + 2); y.w += ld_dyn(a.vec, a.vec_dtype, 4 * g + 3);
      }
      float4 n[S];
#pragma unroll
      for (int t = 0; t < S; ++t) {
        float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int s = 0; s < S; ++s) v = fma4(a.mix[s * S + t], x[k][s], v);
        n[t] = fma4(a.out[t], y, v);
      }
#pragma unroll
      for (int t = 0; t < S; ++t) {
        x[k][t] = n[t];
        if (tid + k * THREADS < n_groups) x4[src + size_t(t) * n_groups + g] = n[t];
      }
    }
  }
  if (!a.h) return;
  float4 u[KEEP];
  double sq = 0.0;
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    u[k] = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int s = 0; s < S; ++s) u[k] = fma4(a.in ? a.in[s] : 1.0f, x[k][s], u[k]);
    if (tid + k * THREADS < n_groups)
      sq += (double(u[k].x * u[k].x) + double(u[k].y * u[k].y)) + (double(u[k].z * u[k].z) + double(u[k].w * u[k].w));
  }
  const float inv = 1.0f / sqrtf(float(block_total<THREADS>(sq) / double(a.width)) + a.eps);
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int g = tid + k * THREADS;
    if (g >= n_groups) continue;
    float o[4] = {u[k].x * inv, u[k].y * inv, u[k].z * inv, u[k].w * inv};
    if (a.w)
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] *= ld_dyn(a.w, a.w_dtype, 4 * g + e);
    const size_t at = size_t(r) * n_groups + g;
    if (a.h_dtype == SB_BF16) {
      uint2 w2;
      w2.x = uint32_t(f32_to_bf16(o[0])) | uint32_t(f32_to_bf16(o[1])) << 16;
      w2.y = uint32_t(f32_to_bf16(o[2])) | uint32_t(f32_to_bf16(o[3])) << 16;
      reinterpret_cast<uint2 *>(a.h)[at] = w2;
    } else {
      reinterpret_cast<float4 *>(a.h)[at] = make_float4(o[0], o[1], o[2], o[3]);
    }
  }
}

// Any width, any number of streams and parts: a column a thread, the read row in LDS.
__global__ void __launch_bounds__(256) streams_any_kernel(StreamArgs a) {
  extern __shared__ float u_row[];
  const int r = blockIdx.x, S = a.streams;
  float *xr = a.x + size_t(a.rows ? a.rows[r] : r) * S * a.width;
  double sq = 0.0;
  for (int c = threadIdx.x; c < a.width; c += 256) {
    float x[kMaxStreams], u = 0.0f;
#pragma unroll
    for (int s = 0; s < kMaxStreams; ++s) x[s] = s < S ? xr[size_t(s) * a.width + c] : 0.0f;
    float y = 0.0f;
    if (a.store) {
      for (int i = 0; i < a.n_parts; ++i) y = fmaf(part_factor(a, i, r), a.part[i][size_t(r) * a.part_stride[i] + c], y);
      if (a.vec) y += ld_dyn(a.vec, a.vec_dtype, c);
    }
    for (int t = 0; t < S; ++t) {
      float v = 0.0f;
      if (a.store) {
#pragma unroll
        for (int s = 0; s < kMaxStreams; ++s)
          if (s < S) v = fmaf(a.mix[s * S + t], x[s], v);
        v = fmaf(a.out[t], y, v);
        xr[size_t(t) * a.width + c] = v;
      } else {
        v = xr[size_t(t) * a.width + c];
      }
      u = fmaf(a.in ? a.in[t] : 1.0f, v, u);
    }
    u_row[c] = u;
    sq += double(u * u);
  }
  if (!a.h) return;
  const float inv = 1.0f / sqrtf(float(block_total<256>(sq) / double(a.width)) + a.eps);
  for (int c = threadIdx.x; c < a.width; c += 256) {
    float o = u_row[c] * inv;
    if (a.w) o *= ld_dyn(a.w, a.w_dtype, c);
    if (a.h_dtype == SB_BF16) ((bf16_t *)a.h)[size_t(r) * a.width + c] = f32_to_bf16(o);
    else ((float *)a.h)[size_t(r) * a.width + c] = o;
  }
}

template <int S, int P>
bool launch_parts(const StreamArgs &a, int n_rows, bool few, hipStream_t s) {
  const int groups = a.width / 4;
  // (a thread's loads are bounded by its registers: two groups of columns where four parts meet four streams)
  constexpr bool two = (S + P) <= 10;
  if (few) {          // few rows: as wide a block as the row fills, so that its loads are one round trip
    if (groups <= 256) streams_kernel<S, P, 256, 1><<<n_rows, 256, 0, s>>>(a);
    else if (groups <= 512) streams_kernel<S, P, 512, 1><<<n_rows, 512, 0, s>>>(a);
    else if (groups <= 1024) streams_kernel<S, P, 1024, 1><<<n_rows, 1024, 0, s>>>(a);
    else return false;
    return true;
  }
  if (groups <= 256) streams_kernel<S, P, 256, 1><<<n_rows, 256, 0, s>>>(a);
  else if (two && groups <= 512) streams_kernel<S, P, 256, two ? 2 : 1><<<n_rows, 256, 0, s>>>(a);
  else if (groups <= 512) streams_kernel<S, P, 512, 1><<<n_rows, 512, 0, s>>>(a);
  else if (two && groups <= 1024) streams_kernel<S, P, 512, two ? 2 : 1><<<n_rows, 512, 0, s>>>(a);
  else if (groups <= 1024) streams_kernel<S, P, 1024, 1><<<n_rows, 1024, 0, s>>>(a);
  else return false;
  return true;
}

template <int S>
bool launch_streams(const StreamArgs &a, int n_rows, bool few, hipStream_t s) {
  if (a.n_parts == 0) return launch_parts<S, 0>(a, n_rows, few, s);
  if (a.n_parts <= 1) return launch_parts<S, 1>(a, n_rows, few, s);
  if (a.n_parts <= 2) return launch_parts<S, 2>(a, n_rows, few, s);
  if (a.n_parts <= 4) return launch_parts<S, 4>(a, n_rows, few, s);
  if (a.n_parts <= 8) return launch_parts<S, 8>(a, n_rows, few, s);
  return launch_parts<S, 16>(a, n_rows, few, s);
}

int launch(const StreamArgs &a, int n_rows, int few, hipStream_t s, const char *what) {
  const auto aligned = [](const void *p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  bool ok = a.width % 4 == 0 && aligned(a.x) && aligned(a.h) && a.n_parts <= 16;
  for (int i = 0; i < a.n_parts; ++i) ok = ok && aligned(a.part[i]) && a.part_stride[i] % 4 == 0;
  if (ok) {
    bool done = false;
    const bool f = few && n_rows <= 64;
    if (a.streams == 1) done = launch_streams<1>(a, n_rows, f, s);
    else if (a.streams == 2) done = launch_streams<2>(a, n_rows, f, s);
    else if (a.streams == 3) done = launch_streams<3>(a, n_rows, f, s);
    else if (a.streams == 4) done = launch_streams<4>(a, n_rows, f, s);
    if (done) return sb::check_launch(what);
  }
  streams_any_kernel<<<n_rows, 256, size_t(a.width) * sizeof(float), s>>>(a);
  return sb::check_launch(what);
}

template <typename T>
__global__ void __launch_bounds__(256)
streams_embed_kernel(float *__restrict__ x, const T *__restrict__ table, const int32_t *__restrict__ ids, int streams, int width,
                     int vocab) {
  const int r = blockIdx.x, id = ids[r];
  const bool ok = id >= 0 && id < vocab;
  float *xr = x + size_t(r) * streams * width;
  for (int c = threadIdx.x; c < width; c += 256) {
    const float v = ok ? ld_f(table, size_t(id) * width + c) : __uint_as_float(0x7fc00000u);
    for (int s = 0; s < streams; ++s) xr[size_t(s) * width + c] = v;
  }
}

}  // namespace

extern "C" int sb_streams_max(void) { return kMaxStreams; }
extern "C" int sb_streams_max_parts(void) { return kMaxSlices; }

extern "C" int sb_streams_embed(float *x, const void *table, int table_dtype, const int32_t *ids, int n_rows, int streams, int width,
                                int vocab, void *stream) {
  SB_REQUIRE(x && table && ids, "sb_streams_embed: null pointer");
  SB_REQUIRE(n_rows >= 0 && streams > 0 && width > 0 && vocab > 0 && sb::valid_dtype(table_dtype),
             "sb_streams_embed: bad sizes rows=%d streams=%d width=%d vocab=%d", n_rows, streams, width, vocab);
  if (n_rows == 0) return SB_OK;
  hipStream_t s = (hipStream_t)stream;
  if (table_dtype == SB_F32) streams_embed_kernel<float><<<n_rows, 256, 0, s>>>(x, (const float *)table, ids, streams, width, vocab);
  else streams_embed_kernel<bf16_t><<<n_rows, 256, 0, s>>>(x, (const bf16_t *)table, ids, streams, width, vocab);
  return sb::check_launch("sb_streams_embed");
}

// Parts: host arrays of n_parts pointers, row strides (in numbers), factors, factors a row (or NULL) and their strides.
// mix f32 [streams][streams] from old to new, out f32 [streams], in f32 [streams] and h with its norm's weight (or
// h NULL: nothing follows).  few: wider blocks for up to 64 rows (the order of a row's sums then depends on the number
// of rows).
extern "C" int sb_streams_join(float *x, const void *const *parts, const int *part_strides, const float *part_scales,
                               const void *const *part_ws, const int *part_w_strides, int n_parts, const void *vec, int vec_dtype,
                               const float *mix, const float *out, const float *in, void *h, int h_dtype, const void *w, int w_dtype,
                               float eps, int n_rows, int streams, int width, int few, void *stream) {
  SB_REQUIRE(x && mix && out && (n_parts == 0 || (parts && part_strides && part_scales && part_ws && part_w_strides)) && (!h || in),
             "sb_streams_join: null pointer");
  SB_REQUIRE(n_rows >= 0 && streams > 0 && width > 0 && n_parts >= 0, "sb_streams_join: bad sizes rows=%d streams=%d width=%d parts=%d",
             n_rows, streams, width, n_parts);
  SB_SUPPORT(streams <= kMaxStreams && n_parts <= kMaxSlices && width <= kMaxWidth,
             "sb_streams_join: %d streams of %d with %d parts are more than %d of %d with %d", streams, width, n_parts, kMaxStreams,
             kMaxWidth, kMaxSlices);
  SB_REQUIRE((!h || sb::valid_dtype(h_dtype)) && (!w || sb::valid_dtype(w_dtype)) && (!vec || sb::valid_dtype(vec_dtype)),
             "sb_streams_join: unknown dtype");
  if (n_rows == 0) return SB_OK;
  StreamArgs a{};
  a.x = x; a.n_parts = n_parts; a.vec = vec; a.vec_dtype = vec_dtype; a.mix = mix; a.out = out; a.in = in;
  a.h = h; a.h_dtype = h_dtype; a.w = w; a.w_dtype = w_dtype; a.eps = eps; a.streams = streams; a.width = width; a.store = 1;
  for (int i = 0; i < n_parts; ++i) {
    SB_REQUIRE(parts[i] && part_strides[i] >= width, "sb_streams_join: bad part %d", i);
    a.part[i] = (const float *)parts[i]; a.part_stride[i] = part_strides[i]; a.part_scale[i] = part_scales[i];
    a.part_w[i] = (const float *)part_ws[i]; a.part_w_stride[i] = part_w_strides[i];
  }
  for (int i = n_parts; n_parts > 0 && i < kMaxSlices; ++i) {
    a.part[i] = a.part[n_parts - 1];
    a.part_stride[i] = a.part_stride[n_parts - 1];
  }
  return launch(a, n_rows, few, (hipStream_t)stream, "sb_streams_join");
}

extern "C" int sb_streams_read(void *h, int h_dtype, const float *x, const int32_t *rows, const float *in, const void *w, int w_dtype,
                               float eps, int n_rows, int streams, int width, int few, void *stream) {
  SB_REQUIRE(h && x, "sb_streams_read: null pointer");
  SB_REQUIRE(n_rows >= 0 && streams > 0 && width > 0, "sb_streams_read: bad sizes rows=%d streams=%d width=%d", n_rows, streams, width);
  SB_SUPPORT(streams <= kMaxStreams && width <= kMaxWidth, "sb_streams_read: %d streams of %d are more than %d of %d", streams, width,
             kMaxStreams, kMaxWidth);
  SB_REQUIRE(sb::valid_dtype(h_dtype) && (!w || sb::valid_dtype(w_dtype)), "sb_streams_read: unknown dtype");
  if (n_rows == 0) return SB_OK;
  StreamArgs a{};
  a.x = const_cast<float *>(x); a.rows = rows; a.in = in; a.h = h; a.h_dtype = h_dtype; a.w = w; a.w_dtype = w_dtype; a.eps = eps;
  a.streams = streams; a.width = width; a.store = 0;
  return launch(a, n_rows, few, (hipStream_t)stream, "sb_streams_read");
}
