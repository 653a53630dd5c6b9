// RMS norms over a whole projection.
//
//   sb_rownorm_kv_store   from the float32 rows of a stacked product [q: heads_q x dk | k: heads_kv x dk |
//       v: heads_kv x dv] (whole, or in K slices that are added here in ascending order): all of q divided by its root
//       mean square over the row (eps inside the root) times a weight as long as q, all of k likewise, then the pairs
//       (i, i + rot_dims / 2) of every head's first rot_dims numbers turned by position * inv_freq[i]; q out in the
//       activation type, k and v into the page of the row's position.
//   sb_rownorm_gate       out = o / rms(o) * w * sigmoid(g), o and g rows of one width (g in K slices or whole).
//
// A block a row; sums of squares in double, per thread in ascending order, a fixed butterfly over the wave, the waves in
// ascending order.
#include "common.h"

namespace {

constexpr int kMaxHalf = 256;          // rotated pairs of a head
constexpr int kMaxRow = 15360;         // numbers of q and k together (they lie in LDS)

struct KVArgs {
  void *q_out;
  const float *qkv; int row_stride, n_slices; size_t slice_stride;
  const void *q_w, *k_w; int w_dtype; float eps;
  const float *inv_freq; int half;
  const int32_t *row_pos, *row_seq, *page_table; int max_pages, n_pages;
  void *k_cache, *v_cache;
  int heads_q, heads_kv, dk, dv;
  int w_eights;                        // bfloat16 weights that are read eight at a time, pairs in eights
};

template <int THREADS, int N>
__device__ __forceinline__ void block_totals(double (&v)[N]) {
  __shared__ double slots[THREADS / 64][N];
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

// number i of the row of q and k after its norm
__device__ __forceinline__ float normed(const KVArgs &a, const float *row, int qw, int i, float q_inv, float k_inv) {
  return i < qw ? (row[i] * q_inv) * ld_dyn(a.q_w, a.w_dtype, i) : (row[i] * k_inv) * ld_dyn(a.k_w, a.w_dtype, i - qw);
}

// and after its pair has turned
__device__ __forceinline__ float turned(const KVArgs &a, const float *row, int qw, int i, int d, float q_inv, float k_inv,
                                        const float *cs, const float *sn) {
  const float v = normed(a, row, qw, i, q_inv, k_inv);
  if (d >= 2 * a.half) return v;
  const bool lo = d < a.half;
  const int p = lo ? d : d - a.half;
  const float o = normed(a, row, qw, lo ? i + a.half : i - a.half, q_inv, k_inv);
  float y0, y1;
  rotate_pair(lo ? v : o, lo ? o : v, cs[p], sn[p], y0, y1);
  return lo ? y0 : y1;
}

__device__ __forceinline__ void lds8(const float *p, float (&v)[8]) {
  const float4 a = reinterpret_cast<const float4 *>(p)[0], b = reinterpret_cast<const float4 *>(p)[1];
  v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
}

// numbers i .. i + 7 of the row of q and k after their norm (bfloat16 weights in eights), as normed() gives them one by one
__device__ __forceinline__ void normed8(const KVArgs &a, const float *row, int qw, int i, float q_inv, float k_inv, float (&v)[8]) {
  const bool is_q = i < qw;
  const uint4 w = *reinterpret_cast<const uint4 *>(is_q ? (const bf16_t *)a.q_w + i : (const bf16_t *)a.k_w + (i - qw));
  const uint32_t u[4] = {w.x, w.y, w.z, w.w};
  const float inv = is_q ? q_inv : k_inv;
  lds8(row + i, v);
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    v[2 * e] = (v[2 * e] * inv) * __uint_as_float(u[e] << 16);
    v[2 * e + 1] = (v[2 * e + 1] * inv) * __uint_as_float(u[e] & 0xffff0000u);
  }
}

// EIGHTS: bfloat16 queries and cache, head sizes in eights: eight numbers a store; FOURS: the row is read four at a time
template <typename TQ, typename TC, int THREADS, bool EIGHTS, bool FOURS>
__global__ void __launch_bounds__(THREADS) rownorm_kv_store_kernel(KVArgs a) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ __attribute__((aligned(16))) float cs[kMaxHalf], sn[kMaxHalf];
  const int r = blockIdx.x, tid = threadIdx.x;
  const float *src = a.qkv + size_t(r) * a.row_stride;
  const int qw = a.heads_q * a.dk, kw = a.heads_kv * a.dk, n = qw + kw;
  const int pos = a.row_pos[r];
  for (int j = tid; j < 2 * a.half; j += THREADS) {
    const int i = j < a.half ? j : j - a.half;
    const float theta = float(pos) * a.inv_freq[i];
    if (j < a.half) cs[i] = cosf(theta);
    else sn[i] = sinf(theta);
  }
  double sq[2] = {0.0, 0.0};
  if (FOURS) {
    for (int i = 4 * tid; i < n; i += 4 * THREADS) {      // (qw is a multiple of four: a four is all q or all k)
      float4 v = *reinterpret_cast<const float4 *>(src + i);
      for (int s = 1; s < a.n_slices; ++s) {
        const float4 p = *reinterpret_cast<const float4 *>(src + s * a.slice_stride + i);
        v.x += p.x; v.y += p.y; v.z += p.z; v.w += p.w;
      }
      *reinterpret_cast<float4 *>(row + i) = v;
      const double t = (double(v.x * v.x) + double(v.y * v.y)) + (double(v.z * v.z) + double(v.w * v.w));
      if (i < qw) sq[0] += t;
      else sq[1] += t;
    }
  } else {
    for (int i = tid; i < n; i += THREADS) {
      const float v = sum_slices(src + i, a.n_slices, a.slice_stride);
      row[i] = v;
      if (i < qw) sq[0] += double(v * v);
      else sq[1] += double(v * v);
    }
  }
  block_totals<THREADS>(sq);
  const float q_inv = 1.0f / sqrtf(float(sq[0] / double(qw)) + a.eps), k_inv = 1.0f / sqrtf(float(sq[1] / double(kw)) + a.eps);
  const int c = pos / SB_PAGE, slot = pos % SB_PAGE;
  int page = c < a.max_pages ? a.page_table[size_t(a.row_seq[r]) * a.max_pages + c] : -1;
  if (page >= a.n_pages) page = -1;
  if (EIGHTS) {
    for (int g = tid; g < n / 8; g += THREADS) {
      const int i0 = 8 * g, head = i0 / a.dk, d0 = i0 - head * a.dk;
      float v[8];
      if (a.w_eights) {                  // (the pairs in eights too: eight numbers turn together, or none does)
        normed8(a, row, qw, i0, q_inv, k_inv, v);
        if (d0 < 2 * a.half) {
          const bool lo = d0 < a.half;
          float o[8], c8[8], s8[8];
          normed8(a, row, qw, lo ? i0 + a.half : i0 - a.half, q_inv, k_inv, o);
          lds8(cs + (lo ? d0 : d0 - a.half), c8);
          lds8(sn + (lo ? d0 : d0 - a.half), s8);
#pragma unroll
          for (int e = 0; e < 8; ++e) {
            float y0, y1;
            rotate_pair(lo ? v[e] : o[e], lo ? o[e] : v[e], c8[e], s8[e], y0, y1);
            v[e] = lo ? y0 : y1;
          }
        }
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = turned(a, row, qw, i0 + e, d0 + e, q_inv, k_inv, cs, sn);
      }
      uint32_t packed[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) packed[e] = uint32_t(f32_to_bf16(v[2 * e])) | uint32_t(f32_to_bf16(v[2 * e + 1])) << 16;
      const uint4 o = make_uint4(packed[0], packed[1], packed[2], packed[3]);
      if (i0 < qw) *reinterpret_cast<uint4 *>((bf16_t *)a.q_out + size_t(r) * qw + i0) = o;
      else if (page >= 0)      // eight neighbouring numbers of a key stay neighbours in the cache's order
        *reinterpret_cast<uint4 *>((bf16_t *)a.k_cache + (size_t(page) * a.heads_kv + (head - a.heads_q)) * SB_PAGE * a.dk +
                                   sb_key_index(slot, d0, a.dk)) = o;
    }
  } else {
    for (int i = tid; i < n; i += THREADS) {
      const int head = i / a.dk, d = i - head * a.dk;
      const float o = turned(a, row, qw, i, d, q_inv, k_inv, cs, sn);
      if (i < qw) st_f((TQ *)a.q_out, size_t(r) * qw + i, o);
      else if (page >= 0)
        st_f((TC *)a.k_cache, (size_t(page) * a.heads_kv + (head - a.heads_q)) * SB_PAGE * a.dk + sb_key_index(slot, d, a.dk), o);
    }
  }
  if (page < 0) return;
  const int nv = a.heads_kv * a.dv;
  for (int e = tid; e < nv; e += THREADS)
    st_f((TC *)a.v_cache, (size_t(page) * a.heads_kv + e / a.dv) * a.dv * SB_PAGE + sb_value_index(e % a.dv, slot),
         sum_slices(src + n + e, a.n_slices, a.slice_stride));
}

template <typename TQ, typename TC, int THREADS, bool EIGHTS>
void launch_store(const KVArgs &a, int n_rows, bool fours, hipStream_t s) {
  const size_t lds = size_t(a.heads_q + a.heads_kv) * a.dk * sizeof(float);
  if (fours) rownorm_kv_store_kernel<TQ, TC, THREADS, EIGHTS, true><<<n_rows, THREADS, lds, s>>>(a);
  else rownorm_kv_store_kernel<TQ, TC, THREADS, EIGHTS, false><<<n_rows, THREADS, lds, s>>>(a);
}

struct GateArgs {
  void *out; int out_dtype;
  const float *o; const void *w; int w_dtype; float eps;
  const float *g; int g_stride, n_slices; size_t slice_stride;
  int width;
};

__device__ __forceinline__ float sigmoid_f(float v) { return 1.0f / (1.0f + expf(-v)); }

// KEEP groups of four a thread (0: a number at a time, any width)
template <int THREADS, int KEEP>
__global__ void __launch_bounds__(THREADS) rownorm_gate_kernel(GateArgs a) {
  const int r = blockIdx.x, tid = threadIdx.x;
  const float *o = a.o + size_t(r) * a.width, *g = a.g + size_t(r) * a.g_stride;
  double sq[1] = {0.0};
  if constexpr (KEEP > 0) {
    const int n = a.width / 4;
    float4 v[KEEP], gt[KEEP];
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
      const int i = min(tid + k * THREADS, n - 1);
      v[k] = reinterpret_cast<const float4 *>(o)[i];
      gt[k] = *reinterpret_cast<const float4 *>(g + 4 * i);
      for (int s = 1; s < a.n_slices; ++s) {
        const float4 p = *reinterpret_cast<const float4 *>(g + s * a.slice_stride + 4 * i);
        gt[k].x += p.x; gt[k].y += p.y; gt[k].z += p.z; gt[k].w += p.w;
      }
      if (tid + k * THREADS < n)
        sq[0] += (double(v[k].x * v[k].x) + double(v[k].y * v[k].y)) + (double(v[k].z * v[k].z) + double(v[k].w * v[k].w));
    }
    block_totals<THREADS>(sq);
    const float inv = 1.0f / sqrtf(float(sq[0] / double(a.width)) + a.eps);
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
      const int i = tid + k * THREADS;
      if (i >= n) continue;
      float y[4] = {v[k].x, v[k].y, v[k].z, v[k].w};
      const float z[4] = {gt[k].x, gt[k].y, gt[k].z, gt[k].w};
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        y[e] *= inv;
        if (a.w) y[e] *= ld_dyn(a.w, a.w_dtype, 4 * i + e);
        y[e] *= sigmoid_f(z[e]);
      }
      const size_t at = size_t(r) * n + i;
      if (a.out_dtype == SB_BF16) {
        uint2 w2;
        w2.x = uint32_t(f32_to_bf16(y[0])) | uint32_t(f32_to_bf16(y[1])) << 16;
        w2.y = uint32_t(f32_to_bf16(y[2])) | uint32_t(f32_to_bf16(y[3])) << 16;
        reinterpret_cast<uint2 *>(a.out)[at] = w2;
      } else {
        reinterpret_cast<float4 *>(a.out)[at] = make_float4(y[0], y[1], y[2], y[3]);
      }
    }
  } else {
    for (int i = tid; i < a.width; i += THREADS) sq[0] += double(o[i] * o[i]);
    block_totals<THREADS>(sq);
    const float inv = 1.0f / sqrtf(float(sq[0] / double(a.width)) + a.eps);
    for (int i = tid; i < a.width; i += THREADS) {
      float y = o[i] * inv;
      if (a.w) y *= ld_dyn(a.w, a.w_dtype, i);
      y *= sigmoid_f(sum_slices(g + i, a.n_slices, a.slice_stride));
      if (a.out_dtype == SB_BF16) ((bf16_t *)a.out)[size_t(r) * a.width + i] = f32_to_bf16(y);
      else ((float *)a.out)[size_t(r) * a.width + i] = y;
    }
  }
}

}  // namespace

extern "C" int sb_rownorm_kv_store(void *q_out, int q_dtype, const float *qkv, int row_stride, int n_slices, size_t slice_stride,
                                   const void *q_w, const void *k_w, int w_dtype, float eps, const float *inv_freq, int rot_dims,
                                   const int32_t *row_pos, const int32_t *row_seq, void *k_cache, void *v_cache, int cache_dtype,
                                   const int32_t *page_table, int max_pages, int n_pages, int n_rows, int heads_q, int heads_kv,
                                   int dk, int dv, void *stream) {
  SB_REQUIRE(q_out && qkv && q_w && k_w && row_pos && row_seq && k_cache && v_cache && page_table, "sb_rownorm_kv_store: null pointer");
  SB_REQUIRE(n_rows >= 0 && heads_q > 0 && heads_kv > 0 && dk > 0 && dv > 0 && n_slices > 0 && max_pages > 0 && n_pages > 0,
             "sb_rownorm_kv_store: bad sizes rows=%d heads=%d/%d dk=%d dv=%d", n_rows, heads_q, heads_kv, dk, dv);
  SB_REQUIRE(row_stride >= heads_q * dk + heads_kv * (dk + dv), "sb_rownorm_kv_store: rows of %d are too short", row_stride);
  SB_REQUIRE(!inv_freq || (rot_dims > 0 && rot_dims % 2 == 0 && rot_dims <= dk),
             "sb_rownorm_kv_store: rotary width %d must be even and at most the head's %d", rot_dims, dk);
  SB_REQUIRE(sb::valid_dtype(q_dtype) && sb::valid_dtype(cache_dtype) && sb::valid_dtype(w_dtype), "sb_rownorm_kv_store: unknown dtype");
  const int n = (heads_q + heads_kv) * dk, half = inv_freq ? rot_dims / 2 : 0;
  SB_SUPPORT(n <= kMaxRow && half <= kMaxHalf, "sb_rownorm_kv_store: %d numbers of queries and keys (%d pairs a head) are more than %d (%d)",
             n, half, kMaxRow, kMaxHalf);
  if (n_rows == 0) return SB_OK;
  const KVArgs a{q_out, qkv, row_stride, n_slices, slice_stride, q_w, k_w, w_dtype, eps, inv_freq, half, row_pos, row_seq, page_table,
                 max_pages, n_pages, k_cache, v_cache, heads_q, heads_kv, dk, dv,
                 w_dtype == SB_BF16 && half % 8 == 0 && ((reinterpret_cast<uintptr_t>(q_w) | reinterpret_cast<uintptr_t>(k_w)) & 15) == 0};
  hipStream_t s = (hipStream_t)stream;
  const auto aligned = [](const void *p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  const bool fours = dk % 4 == 0 && row_stride % 4 == 0 && slice_stride % 4 == 0 && aligned(qkv);
  const bool qf = q_dtype == SB_F32, cf = cache_dtype == SB_F32;
  if (qf && cf) launch_store<float, float, 256, false>(a, n_rows, fours, s);      // (one shape for all row counts)
  else if (qf) launch_store<float, bf16_t, 256, false>(a, n_rows, fours, s);
  else if (cf) launch_store<bf16_t, float, 256, false>(a, n_rows, fours, s);
  else {
    const bool eights = dk % 8 == 0 && aligned(q_out) && aligned(k_cache);
    if (n_rows <= 64) {
      if (eights) launch_store<bf16_t, bf16_t, 1024, true>(a, n_rows, fours, s);
      else launch_store<bf16_t, bf16_t, 1024, false>(a, n_rows, fours, s);
    } else {
      if (eights) launch_store<bf16_t, bf16_t, 256, true>(a, n_rows, fours, s);
      else launch_store<bf16_t, bf16_t, 256, false>(a, n_rows, fours, s);
    }
  }
  return sb::check_launch("sb_rownorm_kv_store");
}

extern "C" int sb_rownorm_gate(void *out, int out_dtype, const float *o, const void *w, int w_dtype, float eps, const float *g,
                               int g_stride, int n_slices, size_t slice_stride, int n_rows, int width, void *stream) {
  SB_REQUIRE(out && o && g, "sb_rownorm_gate: null pointer");
  SB_REQUIRE(n_rows >= 0 && width > 0 && n_slices > 0 && g_stride >= width, "sb_rownorm_gate: bad sizes rows=%d width=%d", n_rows, width);
  SB_REQUIRE(sb::valid_dtype(out_dtype) && (!w || sb::valid_dtype(w_dtype)), "sb_rownorm_gate: unknown dtype");
  if (n_rows == 0) return SB_OK;
  const GateArgs a{out, out_dtype, o, w, w_dtype, eps, g, g_stride, n_slices, slice_stride, width};
  hipStream_t s = (hipStream_t)stream;
  const auto aligned = [](const void *p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  const bool fours = width % 4 == 0 && g_stride % 4 == 0 && slice_stride % 4 == 0 && aligned(out) && aligned(o) && aligned(g);
  if (fours && width <= 1024) rownorm_gate_kernel<256, 1><<<n_rows, 256, 0, s>>>(a);
  else if (fours && width <= 2048) rownorm_gate_kernel<512, 1><<<n_rows, 512, 0, s>>>(a);
  else if (fours && width <= 4096) rownorm_gate_kernel<1024, 1><<<n_rows, 1024, 0, s>>>(a);
  else if (fours && width <= 8192) rownorm_gate_kernel<1024, 2><<<n_rows, 1024, 0, s>>>(a);
  else rownorm_gate_kernel<1024, 0><<<n_rows, 1024, 0, s>>>(a);
  return sb::check_launch("sb_rownorm_gate");
}
