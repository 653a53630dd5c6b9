// Linear attention whose memory of a sequence is a float32 matrix per head that decays from row to row
// without a delta rule:
//     S_t = diag(alpha_t) S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t,          (S is D x E per head)
//     out_t = o_t / sqrt(mean(o_t^2) + eps) (* w) * silu(g_t)
// with alpha either one constant number per head (`decay`) or a number per head and key channel, given by its
// logarithm (`log_decay` [rows, heads * D]) or made here as sb_log_decay makes it from `inner` [rows, rank].  q and k are read from float32 rows; with inv_freq the pairs
// (i, i + rot_dims / 2) of the first rot_dims numbers of every head turn by position * inv_freq[i]; then they are
// multiplied by q_scale and k_scale.  With `act_in` q, k and v are the silu of what is read (before anything turns); with
// `plain` out is o itself, float32, and g is not read.  The state of sequence s lies in state[slots[s]] and goes from step to step.
//
// The walk: a block a (sequence, head), rows in order.  A wave holds NT rows of S for 64 neighbouring columns
// in registers (its loads and stores of the state are whole lines); up to sixteen waves share a head.  Eight rows
// at a time are staged in LDS (queries, keys and decays, which all lanes of a wave then read at one address);
// every wave leaves its share of a row's o in LDS, and after the eight rows a wave a row adds the shares in
// ascending order, norms, gates and stores.  Every number of a row is computed by the same operations in the
// same order whatever the step it came in.
//
// sb_log_decay makes the logarithms: out[r, c] = -softplus(-(sum_j a[r, j] w[j, c] + b[c])) * rate, the logarithm
// of sigmoid(z)^rate, in float32.
#include "common.h"

namespace {

constexpr int RB = 8;              // rows staged in LDS at a time
constexpr int MAX_SIDE = 256;      // rows and columns of a head's matrix at most
constexpr int MAX_WAVES = 16;
constexpr int MAX_RANK = 256;      // inner numbers of a decay that the walk takes

__device__ __forceinline__ float silu_f(float v) { return v / (1.0f + expf(-v)); }

// rate * log(sigmoid(z)) = rate * (min(z, 0) - log(1 + e)), e = exp(-|z|), by log(1 + e) = 2 artanh(s), s = e / (2 + e)
// <= 1/3: 2 (s + s^3/3 + s^5/5 + ..), whose terms from s^17 on are below a float32 result's last digit.
// (The hardware's exponential and reciprocal are right to a few units of the last digit, and e is small where |z| is large.)
__device__ __forceinline__ float log_sigmoid(float z, float rate) {
  const float e = __builtin_amdgcn_exp2f(-fabsf(z) * 1.4426950408889634f), s = e * __builtin_amdgcn_rcpf(2.0f + e), s2 = s * s;
  float p = 1.0f / 15.0f;
  p = fmaf(p, s2, 1.0f / 13.0f);
  p = fmaf(p, s2, 1.0f / 11.0f);
  p = fmaf(p, s2, 1.0f / 9.0f);
  p = fmaf(p, s2, 1.0f / 7.0f);
  p = fmaf(p, s2, 1.0f / 5.0f);
  p = fmaf(p, s2, 1.0f / 3.0f);
  return (fminf(z, 0.0f) - 2.0f * fmaf(s * s2, p, s)) * rate;
}

struct DecayArgs {
  void *out; int out_dtype, out_stride;                  // out_t[a * E + e]
  const float *q, *k, *v, *g; int row_stride;            // q_t[a * D + d], k_t[a * D + d], v_t[a * E + e], g_t[a * E + e]
  int n_slices; size_t slice_stride;                     // (and inner): slices of the rows, added here
  const float *log_decay; int ld_stride;                 // [rows, heads * D], or NULL: inner, or decay
  const float *inner; int inner_stride;                  // [rows, rank]: log alpha = rate log(sigmoid(inner up + bias))
  const float *up, *bias; int rank; float rate;          // [rank, heads * D], [heads * D]
  const float *decay;                                    // [heads]
  const float *inv_freq; int rot_dims; const int32_t *row_pos;
  float q_scale, k_scale;
  const void *w; int w_dtype;                            // [E] or NULL
  float eps;
  float *state;                                          // [slots, heads, D, E]
  const int32_t *cu_rows, *slots;
  int heads, D, E;
  int act_in, plain;                                     // silu on q, k and v; out is o as it is
};

// Column groups of 64 and the rows of S that a wave takes.
template <int NT, bool CHANNEL>
__global__ void __launch_bounds__(1024) decay_walk_kernel(DecayArgs a, int col_groups) {
  __shared__ __attribute__((aligned(16))) float qs[RB][MAX_SIDE], ks[RB][MAX_SIDE], as[CHANNEL ? RB : 1][CHANNEL ? MAX_SIDE : 4], ins[CHANNEL ? RB : 1][CHANNEL ? MAX_RANK : 4];
  __shared__ float vs[RB][MAX_SIDE], gs[RB][MAX_SIDE], os[RB][MAX_WAVES * 64];
  const int head = blockIdx.x, seq = blockIdx.y, tid = threadIdx.x, lane = tid & 63, waves = blockDim.x >> 6;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);      // (the same for all lanes: rows of S are tested once a wave)
  const int cg = wave % col_groups, d0 = (wave / col_groups) * NT, col = cg * 64 + lane;
  const int splits = waves / col_groups, padded = splits * NT;
  const int r0 = a.cu_rows[seq], r1 = a.cu_rows[seq + 1];
  if (r1 <= r0) return;
  float *sp = a.state + (size_t(a.slots[seq]) * a.heads + head) * a.D * a.E;
  float S[NT];
  // rows past the matrix's last read the last again and count as zeros
  const float *from = sp + min(col, a.E - 1);
#pragma unroll
  for (int d = 0; d < NT; ++d) S[d] = from[size_t(min(d0 + d, a.D - 1)) * a.E];
#pragma unroll
  for (int d = 0; d < NT; ++d)
    if (d0 + d >= a.D) S[d] = 0.0f;
  const float fixed = CHANNEL ? 1.0f : a.decay[head];
  const int half = a.inv_freq ? a.rot_dims / 2 : 0;
  for (int rb = r0; rb < r1; rb += RB) {
    const int nr = min(RB, r1 - rb);
    __syncthreads();
    if (CHANNEL && a.inner) {
      for (int idx = tid; idx < nr * a.rank; idx += blockDim.x) {
        const int i = idx / a.rank, j = idx - i * a.rank;
        ins[i][j] = sum_slices(a.inner + size_t(rb + i) * a.inner_stride + j, a.n_slices, a.slice_stride);
      }
      __syncthreads();
    }
    for (int idx = tid; idx < nr * padded; idx += blockDim.x) {
      const int i = idx / padded, d = idx - i * padded;
      const size_t at = size_t(rb + i) * a.row_stride + head * a.D + d;
      float q = 0.0f, k = 0.0f;
      if (d < a.D) {
        q = sum_slices(a.q + at, a.n_slices, a.slice_stride);
        k = sum_slices(a.k + at, a.n_slices, a.slice_stride);
        if (a.act_in) { q = silu_f(q); k = silu_f(k); }
        if (d < 2 * half) {
          const int pair = d < half ? d : d - half, other = d < half ? half : -half;
          const float theta = float(a.row_pos[rb + i]) * a.inv_freq[pair];
          const float c = cosf(theta), s = sinf(theta);
          float y0, y1;
          float qo = sum_slices(a.q + at + other, a.n_slices, a.slice_stride);
          float ko = sum_slices(a.k + at + other, a.n_slices, a.slice_stride);
          if (a.act_in) { qo = silu_f(qo); ko = silu_f(ko); }
          rotate_pair(d < half ? q : qo, d < half ? qo : q, c, s, y0, y1);
          q = d < half ? y0 : y1;
          rotate_pair(d < half ? k : ko, d < half ? ko : k, c, s, y0, y1);
          k = d < half ? y0 : y1;
        }
        q *= a.q_scale;
        k *= a.k_scale;
      }
      qs[i][d] = q;
      ks[i][d] = k;
    }
    if (CHANNEL) {
      // by other waves than those with the first queries and keys, where the block has as many
      for (int idx = tid >= blockDim.x / 2 ? tid - blockDim.x / 2 : tid + (blockDim.x + 1) / 2; idx < nr * padded; idx += blockDim.x) {
        const int i = idx / padded, d = idx - i * padded;
        float al = 1.0f;
        if (d < a.D) {
          float ld;
          if (a.log_decay) {
            ld = a.log_decay[size_t(rb + i) * a.ld_stride + head * a.D + d];
          } else {
            const float *up = a.up + head * a.D + d;
            float z = 0.0f;
#pragma unroll 8
            for (int j = 0; j < a.rank; ++j) z = fmaf(ins[i][j], up[size_t(j) * a.heads * a.D], z);
            ld = log_sigmoid(z + a.bias[head * a.D + d], a.rate);
          }
          al = expf(ld);
        }
        as[i][d] = al;
      }
    }
    for (int idx = tid; idx < nr * a.E; idx += blockDim.x) {
      const int i = idx / a.E, e = idx - i * a.E;
      const size_t at = size_t(rb + i) * a.row_stride + head * a.E + e;
      const float v = sum_slices(a.v + at, a.n_slices, a.slice_stride);
      vs[i][e] = a.act_in ? silu_f(v) : v;
      if (!a.plain) gs[i][e] = silu_f(sum_slices(a.g + at, a.n_slices, a.slice_stride));
    }
    __syncthreads();
#pragma unroll 1
    for (int i = 0; i < nr; ++i) {
      const float v = col < a.E ? vs[i][col] : 0.0f;
      float o = 0.0f;
#pragma unroll
      for (int d = 0; d < NT; d += 4) {
        const float4 k4 = *(const float4 *)&ks[i][d0 + d], q4 = *(const float4 *)&qs[i][d0 + d];
        float4 a4 = make_float4(fixed, fixed, fixed, fixed);
        if (CHANNEL) a4 = *(const float4 *)&as[CHANNEL ? i : 0][CHANNEL ? d0 + d : 0];
        S[d] = fmaf(a4.x, S[d], k4.x * v);             o = fmaf(S[d], q4.x, o);
        S[d + 1] = fmaf(a4.y, S[d + 1], k4.y * v);     o = fmaf(S[d + 1], q4.y, o);
        S[d + 2] = fmaf(a4.z, S[d + 2], k4.z * v);     o = fmaf(S[d + 2], q4.z, o);
        S[d + 3] = fmaf(a4.w, S[d + 3], k4.w * v);     o = fmaf(S[d + 3], q4.w, o);
      }
      os[i][wave * 64 + lane] = o;
    }
    __syncthreads();
    // a wave a row: the waves' shares added in ascending order of S's rows, the norm, the gate, the store
    for (int i = wave; i < nr; i += waves) {
      float o[MAX_SIDE / 64];
      float sq = 0.0f;
#pragma unroll
      for (int c = 0; c < MAX_SIDE / 64; ++c) {
        o[c] = 0.0f;
        if (c < col_groups && c * 64 + lane < a.E) {
          for (int s = 0; s < splits; ++s) o[c] += os[i][(s * col_groups + c) * 64 + lane];
          sq = fmaf(o[c], o[c], sq);
        }
      }
      const float inv = a.plain ? 1.0f : 1.0f / sqrtf(wave_sum(sq) / float(a.E) + a.eps);
#pragma unroll
      for (int c = 0; c < MAX_SIDE / 64; ++c) {
        const int e = c * 64 + lane;
        if (c < col_groups && e < a.E) {
          if (a.plain) {
            ((float *)a.out)[size_t(rb + i) * a.out_stride + head * a.E + e] = o[c];
            continue;
          }
          float y = o[c] * inv;
          if (a.w) y *= ld_dyn(a.w, a.w_dtype, e);
          y *= gs[i][e];
          const size_t at = size_t(rb + i) * a.out_stride + head * a.E + e;
          if (a.out_dtype == SB_F32) ((float *)a.out)[at] = y;
          else ((bf16_t *)a.out)[at] = f32_to_bf16(y);
        }
      }
    }
  }
  if (col >= a.E) return;
  float *to = sp + size_t(d0) * a.E + col;
  if (d0 + NT <= a.D) {
#pragma unroll
    for (int d = 0; d < NT; ++d) to[size_t(d) * a.E] = S[d];
  } else {
    const int left = a.D - d0;
#pragma unroll
    for (int d = 0; d < NT; ++d)
      if (d < left) to[size_t(d) * a.E] = S[d];
  }
}

template <bool CHANNEL>
void launch_walk(const DecayArgs &a, int n_seqs, hipStream_t s) {
  // as many waves a head as leave each at least four rows of S; sixteen at most
  const int col_groups = (a.E + 63) / 64;
  int nt = 4;
  while (col_groups * ((a.D + nt - 1) / nt) > MAX_WAVES) nt *= 2;
  const int splits = (a.D + nt - 1) / nt;
  const dim3 grid(a.heads, n_seqs);
  const int threads = 64 * col_groups * splits;
  if (nt == 4) decay_walk_kernel<4, CHANNEL><<<grid, threads, 0, s>>>(a, col_groups);
  else if (nt == 8) decay_walk_kernel<8, CHANNEL><<<grid, threads, 0, s>>>(a, col_groups);
  else if (nt == 16) decay_walk_kernel<16, CHANNEL><<<grid, threads, 0, s>>>(a, col_groups);
  else if (nt == 32) decay_walk_kernel<32, CHANNEL><<<grid, threads, 0, s>>>(a, col_groups);
  else decay_walk_kernel<64, CHANNEL><<<grid, threads, 0, s>>>(a, col_groups);
}

constexpr int LD_ROWS = 8;         // rows a block of the log-decay kernel takes

__global__ void __launch_bounds__(256)
log_decay_kernel(float *__restrict__ out, int out_stride, const float *__restrict__ a, int a_stride, const float *__restrict__ w,
                 const float *__restrict__ bias, int n_rows, int rank, int width, float rate) {
  extern __shared__ __attribute__((aligned(16))) float as[];    // [rank][LD_ROWS]: a number's eight rows in two loads
  const int r0 = blockIdx.y * LD_ROWS, nr = min(LD_ROWS, n_rows - r0), c = blockIdx.x * 256 + threadIdx.x;
  for (int idx = threadIdx.x; idx < LD_ROWS * rank; idx += 256) {
    const int i = idx / rank, j = idx - i * rank;
    as[j * LD_ROWS + i] = a[size_t(r0 + min(i, nr - 1)) * a_stride + j];
  }
  __syncthreads();
  if (c >= width) return;
  float z[LD_ROWS];
#pragma unroll
  for (int i = 0; i < LD_ROWS; ++i) z[i] = 0.0f;
#pragma unroll 8
  for (int j = 0; j < rank; ++j) {
    const float wv = w[size_t(j) * width + c];
    const float4 lo = *(const float4 *)&as[j * LD_ROWS], hi = *(const float4 *)&as[j * LD_ROWS + 4];
    z[0] = fmaf(lo.x, wv, z[0]); z[1] = fmaf(lo.y, wv, z[1]); z[2] = fmaf(lo.z, wv, z[2]); z[3] = fmaf(lo.w, wv, z[3]);
    z[4] = fmaf(hi.x, wv, z[4]); z[5] = fmaf(hi.y, wv, z[5]); z[6] = fmaf(hi.z, wv, z[6]); z[7] = fmaf(hi.w, wv, z[7]);
  }
  const float b = bias ? bias[c] : 0.0f;
#pragma unroll
  for (int i = 0; i < LD_ROWS; ++i)
    if (i < nr) {
      out[size_t(r0 + i) * out_stride + c] = log_sigmoid(z[i] + b, rate);
    }
}

}  // namespace

extern "C" int sb_decay_scan_max_side(void) { return MAX_SIDE; }
extern "C" int sb_decay_scan_max_rank(void) { return MAX_RANK; }

extern "C" int sb_decay_scan(void *out, int out_dtype, int out_stride, const float *q, const float *k, const float *v,
                             const float *g, int row_stride, int n_slices, size_t slice_stride,
                             const float *log_decay, int ld_stride, const float *inner,
                             int inner_stride, const float *up, const float *bias, int rank, float rate, const float *decay,
                             const float *inv_freq, int rot_dims, const int32_t *row_pos, float q_scale, float k_scale,
                             const void *w, int w_dtype, float eps, float *state, const int32_t *cu_rows,
                             const int32_t *slots, int n_seqs, int heads, int D, int E, int act_in, int plain, void *stream) {
  SB_REQUIRE(out && q && k && v && (g || plain) && state && cu_rows && slots && (log_decay || inner || decay), "sb_decay_scan: null pointer");
  SB_REQUIRE(!plain || out_dtype == SB_F32, "sb_decay_scan: what is read goes out in float32");
  SB_REQUIRE(!inner || (up && bias && rank > 0), "sb_decay_scan: decays without their matrix or bias");
  SB_SUPPORT(!inner || rank <= MAX_RANK, "sb_decay_scan: a rank of %d is more than %d", rank, MAX_RANK);
  SB_REQUIRE(n_slices >= 1, "sb_decay_scan: at least one slice");
  SB_REQUIRE(n_seqs >= 0 && heads > 0 && D > 0 && E > 0 && sb::valid_dtype(out_dtype) && (!w || sb::valid_dtype(w_dtype)),
             "sb_decay_scan: bad sizes heads=%d dim=%d vdim=%d", heads, D, E);
  SB_REQUIRE(!inv_freq || (row_pos && rot_dims > 0 && rot_dims % 2 == 0 && rot_dims <= D),
             "sb_decay_scan: rotary width %d must be even and at most the head's %d", rot_dims, D);
  SB_SUPPORT(D <= MAX_SIDE && E <= MAX_SIDE, "sb_decay_scan: a state of %d x %d a head is more than %d x %d", D, E, MAX_SIDE, MAX_SIDE);
  SB_SUPPORT(n_seqs <= 65535, "sb_decay_scan: more than 65535 sequences");
  if (n_seqs == 0) return SB_OK;
  const DecayArgs a{out, out_dtype, out_stride, q, k, v, g, row_stride, n_slices, slice_stride, log_decay, ld_stride, inner, inner_stride, up, bias,
                    rank, rate, decay, inv_freq, inv_freq ? rot_dims : 0,
                    row_pos, q_scale, k_scale, w, w_dtype, eps, state, cu_rows, slots, heads, D, E, act_in, plain};
  if (log_decay || inner) launch_walk<true>(a, n_seqs, (hipStream_t)stream);
  else launch_walk<false>(a, n_seqs, (hipStream_t)stream);
  return sb::check_launch("sb_decay_scan");
}

// a f32 [n_rows, a_stride], w f32 [rank, width], bias f32 [width] or NULL, out f32 [n_rows, out_stride].
extern "C" int sb_log_decay(float *out, int out_stride, const float *a, int a_stride, const float *w, const float *bias,
                            int n_rows, int rank, int width, float rate, void *stream) {
  SB_REQUIRE(out && a && w, "sb_log_decay: null pointer");
  SB_REQUIRE(n_rows >= 0 && rank > 0 && width > 0 && a_stride >= rank && out_stride >= width,
             "sb_log_decay: bad sizes rows=%d rank=%d width=%d", n_rows, rank, width);
  SB_SUPPORT(rank <= 1024, "sb_log_decay: a rank of %d is more than 1024", rank);
  SB_SUPPORT(n_rows <= 65535 * LD_ROWS, "sb_log_decay: too many rows");
  if (n_rows == 0) return SB_OK;
  log_decay_kernel<<<dim3((width + 255) / 256, (n_rows + LD_ROWS - 1) / LD_ROWS), 256, size_t(LD_ROWS) * rank * sizeof(float),
                     (hipStream_t)stream>>>(out, out_stride, a, a_stride, w, bias, n_rows, rank, width, rate);
  return sb::check_launch("sb_log_decay");
}
