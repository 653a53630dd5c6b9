// The chunked form of linear attention with decays (decay_scan.hip has the walk and the equations), for long
// prompts: runs ("chunks") of consecutive rows of one sequence on the matrix cores in float32
// (v_mfma_f32_16x16x4_f32), in three launches.  With l_t the logarithm of alpha (a number a key channel, or one a
// head) and L_i its sum over the chunk's rows up to and with row i:
//   LOCAL  a block a (chunk, head): A_c = sum_j (k_j exp(L_last - L_j)) v_j^T, and exp(L_last);
//   carry  a sequence's chunks in order: S_in(c) is put where A_c lay, S_in(c + 1) = exp(L_last) S_in(c) + A_c, and
//          the last one is the sequence's state;
//   FROM   a block a (chunk, head): o_i = (q_i exp(L_i)) S_in + sum_{j <= i} P_ij v_j,
//          P_ij = sum_d q_i[d] k_j[d] exp(L_i[d] - L_j[d]); then the head's norm, the weight, the gate, the store.
// No exponent is positive, however fast a channel decays: with one decay a head P is the plain product q k^T times
// a power of the decay; with a decay a channel a tile of 16 x 16 pairs away from the diagonal takes
// exp(L_i - R) and exp(R - L_j) with R = L at the row before the tile's first row i, and the pairs of a tile on the
// diagonal are summed one by one on the vector units with exp(L_i - L_j) as it is.
//
// With `act_in` q, k and v are the silu of what is read; with `plain` o goes out as it is, float32, and g is not read.
// q and k may turn on the way in, by a table of the rows' cosines and sines (sb_angle_table, once a step).
// Operands in LDS: rows a multiple of 64 numbers and four further on, so that the sixteen rows and four columns a
// wave's operand takes lie in distinct banks; where the rows are summed over, sixteen further on.
#include "common.h"

namespace {

typedef float f32x4_t __attribute__((ext_vector_type(4)));

constexpr int THREADS = 512, WAVES = THREADS / 64;
constexpr float kLog2e = 1.4426950408889634f;
constexpr float kLeastLog = -110.0f;      // exp of it is 0 in float32: sums of a chunk's logarithms keep their digits

__device__ __forceinline__ float exp2_f(float v) { return __builtin_amdgcn_exp2f(v); }
__device__ __forceinline__ f32x4_t mfma_f32(float a, float b, f32x4_t c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

struct ChunkArgs {
  void *out; int out_dtype, out_stride;
  const float *q, *k, *v, *g; int row_stride;
  const float *log_decay; int ld_stride;     // [rows, heads * D], or NULL: decay
  const float *decay;                        // [heads]
  const float2 *angles; int half;            // [rows, half] cosine and sine, or NULL
  float q_scale, k_scale;
  const void *w; int w_dtype;
  float eps;
  float *state;                              // [slots, heads, D, E]
  const int32_t *cu_rows, *slots;
  int heads, D, E;
  const int32_t *chunks;                     // [n_chunks, 4]: first row, rows, sequence, 0
  float *part;                               // [n_chunks, heads, D, E]: A_c, then S_in(c)
  float *part_decay;                         // [n_chunks, heads, D]: exp(L_last) (a decay a channel only)
  int vec4;                                  // rows can be read four numbers at a time
  int act_in, plain;                         // silu on q, k and v; out is o as it is
};

__device__ __forceinline__ float silu_f(float v) { return v / (1.0f + expf(-v)); }

// What a thread needs for four numbers of a head's row: themselves, what they turn with, cosines and sines.
struct Four { float4 x, o, t0, t1; };

// The loads for numbers d .. d + 3 of row `row`; no branch stands between them (numbers past the head's last read its
// last again, heads that do not turn skip the rest).  turning: 2 with their angles, 1 without (asked for before), 0 not.
__device__ __forceinline__ void fetch_four(Four &f, const ChunkArgs &a, const float *head, int row, int d, int turning) {
  const float *src = head + size_t(row) * a.row_stride;
  const int at = min(d, a.D - 4);
  f.x = *(const float4 *)(src + at);
  if (turning) {            // (half is a multiple of 4: the four turn together, or none does)
    const bool lo = at < a.half, on = at < 2 * a.half;
    f.o = *(const float4 *)(src + (on ? (lo ? at + a.half : at - a.half) : at));
    if (turning == 2) {
      const float2 *t = a.angles + size_t(row) * a.half + (on ? (lo ? at : at - a.half) : 0);
      f.t0 = *(const float4 *)t;
      f.t1 = *(const float4 *)(t + 2);
    }
  }
}

__device__ __forceinline__ float4 finish_four(const Four &f, const ChunkArgs &a, int d, bool live, float scale, bool turning) {
  float x[4] = {f.x.x, f.x.y, f.x.z, f.x.w};
  if (a.act_in) {
#pragma unroll
    for (int e = 0; e < 4; ++e) x[e] = silu_f(x[e]);
  }
  if (turning) {
    const bool lo = d < a.half, on = d < 2 * a.half;
    float o[4] = {f.o.x, f.o.y, f.o.z, f.o.w};
    if (a.act_in) {
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] = silu_f(o[e]);
    }
    const float c[4] = {f.t0.x, f.t0.z, f.t1.x, f.t1.z}, s[4] = {f.t0.y, f.t0.w, f.t1.y, f.t1.w};
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      float y0, y1;
      rotate_pair(lo ? x[e] : o[e], lo ? o[e] : x[e], c[e], s[e], y0, y1);
      x[e] = on ? (lo ? y0 : y1) : x[e];
    }
  }
  if (!live || d >= a.D) return make_float4(0.f, 0.f, 0.f, 0.f);
  return make_float4(x[0] * scale, x[1] * scale, x[2] * scale, x[3] * scale);
}

// The same for rows that cannot be read four numbers at a time.
__device__ __forceinline__ float4 load_single(const ChunkArgs &a, const float *head, int row, int d, float scale) {
  const float *src = head + size_t(row) * a.row_stride;
  float x[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    if (d + e >= a.D) continue;
    x[e] = a.act_in ? silu_f(src[d + e]) : src[d + e];
    if (d + e < 2 * a.half) {
      const bool lo = d + e < a.half;
      const int i = lo ? d + e : d + e - a.half;
      float ov = src[lo ? d + e + a.half : d + e - a.half];
      if (a.act_in) ov = silu_f(ov);
      const float2 t = a.angles[size_t(row) * a.half + i];
      float y0, y1;
      rotate_pair(lo ? x[e] : ov, lo ? ov : x[e], t.x, t.y, y0, y1);
      x[e] = lo ? y0 : y1;
    }
    x[e] *= scale;
  }
  return make_float4(x[0], x[1], x[2], x[3]);
}

// The chunk's queries (or NULL) and keys into LDS, rows of STRIDE numbers; rows past the chunk's last are zeros.
template <int DP, int CR, int STRIDE>
__device__ __forceinline__ void stage_heads(const ChunkArgs &a, const float *qp, const float *kp, int r0, int nr, float *qs, float *ks) {
  constexpr int N = CR * (DP / 4) / THREADS;         // fours a thread
  if (a.vec4) {
    const bool turning = a.half > 0;
    Four q[N], k[N];
#pragma unroll
    for (int u = 0; u < N; ++u) {
      const int idx = threadIdx.x + u * THREADS, row = r0 + min(idx / (DP / 4), nr - 1), d = (idx % (DP / 4)) * 4;
      fetch_four(k[u], a, kp, row, d, turning ? 2 : 0);
      if (qp) fetch_four(q[u], a, qp, row, d, turning ? 1 : 0);
    }
#pragma unroll
    for (int u = 0; u < N; ++u) {
      const int idx = threadIdx.x + u * THREADS, i = idx / (DP / 4), d = (idx % (DP / 4)) * 4;
      *(float4 *)&ks[i * STRIDE + d] = finish_four(k[u], a, d, i < nr, a.k_scale, turning);
      if (qp) {
        q[u].t0 = k[u].t0; q[u].t1 = k[u].t1;
        *(float4 *)&qs[i * STRIDE + d] = finish_four(q[u], a, d, i < nr, a.q_scale, turning);
      }
    }
  } else {
    for (int idx = threadIdx.x; idx < CR * (DP / 4); idx += THREADS) {
      const int i = idx / (DP / 4), d = (idx % (DP / 4)) * 4;
      float4 x = make_float4(0.f, 0.f, 0.f, 0.f), y = x;
      if (i < nr) {
        y = load_single(a, kp, r0 + i, d, a.k_scale);
        if (qp) x = load_single(a, qp, r0 + i, d, a.q_scale);
      }
      *(float4 *)&ks[i * STRIDE + d] = y;
      if (qp) *(float4 *)&qs[i * STRIDE + d] = x;
    }
  }
}

// The logarithms of a thread's channel over its part of the chunk's rows (rows past the last read the last again).
template <int PR>
__device__ __forceinline__ void fetch_logs(const ChunkArgs &a, float *l, int head, int r0, int nr, int d, int part) {
  const float *src = a.log_decay + head * a.D + min(d, a.D - 1);
#pragma unroll
  for (int i = 0; i < PR; ++i) l[i] = src[size_t(r0 + min(part * PR + i, nr - 1)) * a.ld_stride];
}

// powers of the head's decay, 0 .. n
__device__ __forceinline__ void decay_powers(float *pow_lds, float decay, int n) {
  const float l = log2f(decay);
  for (int i = threadIdx.x; i <= n; i += THREADS) pow_lds[i] = i == 0 ? 1.0f : exp2_f(float(i) * l);
}

template <int DP, int CR, int EP, bool CHANNEL>
__global__ void __launch_bounds__(THREADS) chunk_local_kernel(ChunkArgs a) {
  constexpr int KS = DP + 16, VS = EP + 16, PARTS = THREADS / DP, PR = CR / PARTS;     // rows of a part
  __shared__ __attribute__((aligned(16))) float ks[CR][KS], vs[CR][VS];
  __shared__ float sums[CHANNEL ? PARTS : 1][CHANNEL ? DP : 1], pw[CR + 1];
  const int head = blockIdx.x, tid = threadIdx.x, lane = tid & 63;
  const int32_t *c = a.chunks + 4 * size_t(blockIdx.y);
  const int r0 = c[0], nr = c[1];
  const float *kp = a.k + size_t(head) * a.D, *vp = a.v + size_t(head) * a.E;
  if (!CHANNEL) decay_powers(pw, a.decay[head], CR);
  // the logarithms are asked for first, then the values, then the keys
  float l[CHANNEL ? PR : 1];
  const int ch = tid % DP, part = tid / DP;
  if (CHANNEL) fetch_logs<PR>(a, l, head, r0, nr, ch, part);
  constexpr int NV = CR * (EP / 4) / THREADS;
  if (a.vec4) {
    float4 x[NV];
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const int idx = tid + u * THREADS, row = r0 + min(idx / (EP / 4), nr - 1), e = (idx % (EP / 4)) * 4;
      x[u] = *(const float4 *)(vp + size_t(row) * a.row_stride + min(e, a.E - 4));
    }
    stage_heads<DP, CR, KS>(a, nullptr, kp, r0, nr, nullptr, &ks[0][0]);
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const int idx = tid + u * THREADS, i = idx / (EP / 4), e = (idx % (EP / 4)) * 4;
      if (a.act_in) x[u] = make_float4(silu_f(x[u].x), silu_f(x[u].y), silu_f(x[u].z), silu_f(x[u].w));
      *(float4 *)&vs[i][e] = (i < nr && e < a.E) ? x[u] : make_float4(0.f, 0.f, 0.f, 0.f);
    }
  } else {
    stage_heads<DP, CR, KS>(a, nullptr, kp, r0, nr, nullptr, &ks[0][0]);
    for (int idx = tid; idx < CR * EP; idx += THREADS) {
      const int i = idx / EP, e = idx % EP;
      float v = (i < nr && e < a.E) ? vp[size_t(r0 + i) * a.row_stride + e] : 0.0f;
      vs[i][e] = a.act_in ? silu_f(v) : v;
    }
  }
  __syncthreads();
  if (CHANNEL) {
    // a thread a (channel, part of the rows): the sum of the logarithms of the rows after a row, backwards
    const int d = ch;
    float total = 0.0f;
#pragma unroll
    for (int i = 0; i < PR; ++i) {
      l[i] = (d < a.D && part * PR + i < nr) ? fmaxf(l[i], kLeastLog) * kLog2e : 0.0f;
      total += l[i];
    }
    sums[part][d] = total;
    __syncthreads();
    float after = 0.0f;
    for (int p = part + 1; p < PARTS; ++p) after += sums[p][d];
#pragma unroll
    for (int i = PR - 1; i >= 0; --i) {
      ks[part * PR + i][d] *= exp2_f(after);
      after += l[i];
    }
    if (part == 0 && d < a.D) a.part_decay[(size_t(blockIdx.y) * a.heads + head) * a.D + d] = exp2_f(after);
  } else {
    for (int idx = tid; idx < nr * DP; idx += THREADS) {
      const int i = idx / DP, d = idx % DP;
      ks[i][d] *= pw[nr - 1 - i];
    }
  }
  __syncthreads();
  // tiles of A_c: a wave a (16 key channels, 64 columns) at a time
  const int wave = tid >> 6, col = lane & 15, grp = lane >> 4;
  const int n_dt = (a.D + 15) / 16, n_eg = (a.E + 63) / 64, steps = (nr + 3) / 4;
  float *dst = a.part + (size_t(blockIdx.y) * a.heads + head) * a.D * a.E;
  for (int item = wave; item < n_dt * n_eg; item += WAVES) {
    const int d0 = (item % n_dt) * 16, e0 = (item / n_dt) * 64;
    f32x4_t acc[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) acc[t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int s = 0; s < steps; ++s) {
      const int j = 4 * s + grp;
      const float kv = ks[j][d0 + col];
#pragma unroll
      for (int t = 0; t < 4; ++t) acc[t] = mfma_f32(kv, vs[j][e0 + 16 * t + col], acc[t]);
    }
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = d0 + 4 * grp + r, e = e0 + 16 * t + col;
        if (d < a.D && e < a.E) dst[size_t(d) * a.E + e] = acc[t][r];
      }
  }
}

// A sequence's chunks in order, a thread an element of the head's matrix.  The chunks' additions are asked for
// eight at a time.
__global__ void __launch_bounds__(256) chunk_carry_kernel(ChunkArgs a, int chunk_rows) {
  constexpr int AHEAD = 8;
  const int head = blockIdx.x, seq = blockIdx.y;
  const int len = a.cu_rows[seq + 1] - a.cu_rows[seq];
  if (len <= 0) return;
  const int size = a.D * a.E, e = blockIdx.z * 256 + threadIdx.x;
  if (e >= size) return;
  const int n = (len + chunk_rows - 1) / chunk_rows, d = e / a.E;
  int c0 = 0;
  for (int s = 0; s < seq; ++s) c0 += (a.cu_rows[s + 1] - a.cu_rows[s] + chunk_rows - 1) / chunk_rows;
  float *sp = a.state + (size_t(a.slots[seq]) * a.heads + head) * size + e;
  float cur = *sp;
  float *pp = a.part + (size_t(c0) * a.heads + head) * size + e;
  const float *dp = a.part_decay ? a.part_decay + (size_t(c0) * a.heads + head) * a.D + d : nullptr;
  const size_t step = size_t(a.heads) * size, dstep = size_t(a.heads) * a.D;
  float fixed = 0.0f;
  if (!dp) fixed = exp2_f(float(chunk_rows) * log2f(a.decay[head]));
  for (int c = 0; c < n; c += AHEAD) {
    float add[AHEAD], dec[AHEAD];
#pragma unroll
    for (int u = 0; u < AHEAD; ++u) {
      const int at = min(u, n - 1 - c);
      add[u] = pp[size_t(at) * step];
      dec[u] = dp ? dp[size_t(at) * dstep] : fixed;
    }
#pragma unroll
    for (int u = 0; u < AHEAD; ++u)
      if (c + u < n) {
        pp[size_t(u) * step] = cur;
        // the last chunk may be short
        if (!dp && c + u == n - 1) dec[u] = exp2_f(float(len - (n - 1) * chunk_rows) * log2f(a.decay[head]));
        cur = fmaf(dec[u], cur, add[u]);
      }
    pp += AHEAD * step;
    if (dp) dp += AHEAD * dstep;
  }
  *sp = cur;
}

// ET: column tiles of 16 a wave takes; RSPLIT: waves that share a column tile, each with its share of the rows
template <int DP, int CR, int ET, int RSPLIT, bool CHANNEL>
__global__ void __launch_bounds__(THREADS) chunk_from_kernel(ChunkArgs a) {
  constexpr int QS = DP + 4, PS = CR + 4, NT = CR / 16, RT = NT / RSPLIT;      // row tiles, and those of a wave
  constexpr int PARTS = THREADS / DP, PR = CR / PARTS;
  constexpr int KP = CR * QS > CR * PS ? CR * QS : CR * PS;
  __shared__ __attribute__((aligned(16))) float qs[CR * QS], kps[KP];          // the keys, then P
  __shared__ __attribute__((aligned(16))) float ls[CHANNEL ? CR * QS : 4], diag[CHANNEL ? NT * 16 * 17 : 4];
  __shared__ float sums[CHANNEL ? PARTS : 1][CHANNEL ? DP : 1], pw[CR + 1], sq[CR][WAVES + 1];
  const int head = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 15, grp = lane >> 4;
  const int32_t *c = a.chunks + 4 * size_t(blockIdx.y);
  const int r0 = c[0], nr = c[1];
  const float *qp = a.q + size_t(head) * a.D, *kp = a.k + size_t(head) * a.D, *vp = a.v + size_t(head) * a.E;
  if (!CHANNEL) decay_powers(pw, a.decay[head], CR);
  float l[CHANNEL ? PR : 1];
  const int ch = tid % DP, part = tid / DP;
  if (CHANNEL) fetch_logs<PR>(a, l, head, r0, nr, ch, part);
  stage_heads<DP, CR, QS>(a, qp, kp, r0, nr, qs, kps);
  // What the second half of the kernel reads from memory is asked for now and arrives while P is made: the wave's
  // columns of S_in, of the chunk's values and of the gate.
  const int rsub = RSPLIT > 1 ? wave / (WAVES / RSPLIT) : 0, ew = RSPLIT > 1 ? wave % (WAVES / RSPLIT) : wave;
  const int t0 = rsub * RT;                                // the wave's first row tile
  const float *S = a.part + (size_t(blockIdx.y) * a.heads + head) * a.D * a.E;
  float sv[ET][DP / 4], vv[ET][CR / 4];
#pragma unroll
  for (int x = 0; x < ET; ++x) {
    const int e = min((ew + x * (WAVES / RSPLIT)) * 16 + col, a.E - 1);
#pragma unroll
    for (int u = 0; u < DP / 4; ++u) sv[x][u] = S[size_t(min(4 * u + grp, a.D - 1)) * a.E + e];
#pragma unroll
    for (int u = 0; u < CR / 4; ++u) vv[x][u] = vp[size_t(r0 + min(4 * u + grp, nr - 1)) * a.row_stride + e];
  }
  if (CHANNEL) {
    // L, times log2(e): a thread a (channel, part of the rows)
    float total = 0.0f;
#pragma unroll
    for (int i = 0; i < PR; ++i) {
      l[i] = (ch < a.D && part * PR + i < nr) ? fmaxf(l[i], kLeastLog) * kLog2e : 0.0f;
      total += l[i];
    }
    sums[part][ch] = total;
    __syncthreads();
    float before = 0.0f;
    for (int p = 0; p < part; ++p) before += sums[p][ch];
#pragma unroll
    for (int i = 0; i < PR; ++i) {
      before += l[i];
      ls[(part * PR + i) * QS + ch] = before;
    }
  }
  __syncthreads();
  // ---- P, tile by tile of its lower triangle: tile (I, J), J <= I
  const int ksteps = (a.D + 3) / 4;
  constexpr int OFF = NT * (NT - 1) / 2, ALL = NT * (NT + 1) / 2;
  constexpr int TILES = CHANNEL ? OFF : ALL, PER_WAVE = (TILES + WAVES - 1) / WAVES;
  f32x4_t pt[PER_WAVE > 0 ? PER_WAVE : 1];
#pragma unroll
  for (int u = 0; u < PER_WAVE; ++u) {
    pt[u] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const int t = wave + u * WAVES;
    if (t >= TILES) continue;
    int I = CHANNEL ? 1 : 0, J = t;                       // rows of tiles hold 1, 2, 3, .. tiles
    while (J >= (CHANNEL ? I : I + 1)) { J -= CHANNEL ? I : I + 1; ++I; }
    const float *qr = qs + (16 * I + col) * QS + grp, *kr = kps + (16 * J + col) * QS + grp;
    if (CHANNEL) {
      const float *li = ls + (16 * I + col) * QS + grp, *lj = ls + (16 * J + col) * QS + grp, *lr = ls + (16 * I - 1) * QS + grp;
#pragma unroll 4
      for (int s = 0; s < ksteps; ++s) {
        const float ref = lr[4 * s];
        pt[u] = mfma_f32(qr[4 * s] * exp2_f(li[4 * s] - ref), kr[4 * s] * exp2_f(ref - lj[4 * s]), pt[u]);
      }
    } else {
#pragma unroll 8
      for (int s = 0; s < ksteps; ++s) pt[u] = mfma_f32(qr[4 * s], kr[4 * s], pt[u]);
    }
  }
  if (CHANNEL) {
    // pairs of the tiles on the diagonal: 128 threads a tile, 120 pairs j < i and eight threads with two i = j each
    constexpr int GROUPS = THREADS / 128;
    const int t = tid & 127;
    for (int tile = tid >> 7; tile < NT; tile += GROUPS) {
      if (t < 120) {
        int i = 1, j = t;
        while (j >= i) { j -= i; ++i; }
        const float *qr = qs + (16 * tile + i) * QS, *kr = kps + (16 * tile + j) * QS;
        const float *li = ls + (16 * tile + i) * QS, *lj = ls + (16 * tile + j) * QS;
        float sum = 0.0f;
#pragma unroll 4
        for (int d = 0; d < 4 * ksteps; d += 4) {
          const float4 q4 = *(const float4 *)(qr + d), k4 = *(const float4 *)(kr + d), a4 = *(const float4 *)(li + d),
                       b4 = *(const float4 *)(lj + d);
          sum = fmaf(q4.x * k4.x, exp2_f(a4.x - b4.x), sum);
          sum = fmaf(q4.y * k4.y, exp2_f(a4.y - b4.y), sum);
          sum = fmaf(q4.z * k4.z, exp2_f(a4.z - b4.z), sum);
          sum = fmaf(q4.w * k4.w, exp2_f(a4.w - b4.w), sum);
        }
        diag[(tile * 16 + i) * 17 + j] = sum;
      } else {
        for (int i = 2 * (t - 120); i < 2 * (t - 120) + 2; ++i) {
          const float *qr = qs + (16 * tile + i) * QS, *kr = kps + (16 * tile + i) * QS;
          float sum = 0.0f;
          for (int d = 0; d < 4 * ksteps; d += 4) {
            const float4 q4 = *(const float4 *)(qr + d), k4 = *(const float4 *)(kr + d);
            sum = fmaf(q4.x, k4.x, fmaf(q4.y, k4.y, fmaf(q4.z, k4.z, fmaf(q4.w, k4.w, sum))));
          }
          diag[(tile * 16 + i) * 17 + i] = sum;
        }
      }
    }
  }
  __syncthreads();          // the keys have been read: P takes their place
  float *ps = kps;
#pragma unroll
  for (int u = 0; u < PER_WAVE; ++u) {
    const int t = wave + u * WAVES;
    if (t >= TILES) continue;
    int I = CHANNEL ? 1 : 0, J = t;
    while (J >= (CHANNEL ? I : I + 1)) { J -= CHANNEL ? I : I + 1; ++I; }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * I + 4 * grp + r, j = 16 * J + col;
      float p = pt[u][r];
      if (!CHANNEL) p = j <= i ? p * pw[max(i - j, 0)] : 0.0f;
      ps[i * PS + j] = p;
    }
  }
  if (CHANNEL) {
    for (int idx = tid; idx < NT * 256; idx += THREADS) {
      const int tile = idx >> 8, i = (idx >> 4) & 15, j = idx & 15;
      ps[(16 * tile + i) * PS + 16 * tile + j] = j <= i ? diag[(tile * 16 + i) * 17 + j] : 0.0f;
    }
    // the queries as the matrix that comes in is read: q_i exp(L_i)
    for (int idx = tid; idx < CR * DP; idx += THREADS) {
      const int i = idx / DP, d = idx % DP;
      qs[i * QS + d] *= exp2_f(ls[i * QS + d]);
    }
  }
  __syncthreads();
  if (a.act_in) {
#pragma unroll
    for (int x = 0; x < ET; ++x)
#pragma unroll
      for (int u = 0; u < CR / 4; ++u) vv[x][u] = silu_f(vv[x][u]);
  }
  // ---- o = q S_in (scaled) + P v
  f32x4_t acc[ET][RT];
  bool live[ET];
#pragma unroll
  for (int x = 0; x < ET; ++x) {
    live[x] = (ew + x * (WAVES / RSPLIT)) * 16 < a.E;
#pragma unroll
    for (int t = 0; t < RT; ++t) acc[x][t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    if (!live[x]) continue;
#pragma unroll
    for (int u = 0; u < DP / 4; ++u) {
      if (u < ksteps)                     // (numbers past the head's last are zeros in the queries)
#pragma unroll
        for (int t = 0; t < RT; ++t) acc[x][t] = mfma_f32(qs[(16 * (t0 + t) + col) * QS + 4 * u + grp], sv[x][u], acc[x][t]);
    }
    if (!CHANNEL) {
#pragma unroll
      for (int t = 0; t < RT; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[x][t][r] *= pw[16 * (t0 + t) + 4 * grp + r + 1];
    }
    // the chunk's own rows: column tile J of P meets rows 16 J .. of v; row tiles before J have none of it
#pragma unroll
    for (int J = 0; J < NT; ++J)
#pragma unroll
      for (int t = 0; t < RT; ++t) {
        if (t0 + t < J) continue;         // uniform over the wave
#pragma unroll
        for (int s = 0; s < 4; ++s)
          acc[x][t] = mfma_f32(ps[(16 * (t0 + t) + col) * PS + 16 * J + 4 * s + grp], vv[x][4 * J + s], acc[x][t]);
      }
  }
  if (a.plain) {
#pragma unroll
    for (int x = 0; x < ET; ++x) {
      const int e = (ew + x * (WAVES / RSPLIT)) * 16 + col;
      if (!live[x] || e >= a.E) continue;
#pragma unroll
      for (int t = 0; t < RT; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int i = 16 * (t0 + t) + 4 * grp + r;
          if (i < nr) ((float *)a.out)[size_t(r0 + i) * a.out_stride + head * a.E + e] = acc[x][t][r];
        }
    }
    return;
  }
  // the gate's numbers arrive while the norms are worked out
  float gate[ET][RT][4];
#pragma unroll
  for (int x = 0; x < ET; ++x) {
    const int e = min((ew + x * (WAVES / RSPLIT)) * 16 + col, a.E - 1);
#pragma unroll
    for (int t = 0; t < RT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        gate[x][t][r] = a.g[size_t(r0 + min(16 * (t0 + t) + 4 * grp + r, nr - 1)) * a.row_stride + head * a.E + e];
  }
  // ---- the head's norm: a row's squares over the sixteen lanes, then over the waves that share it
#pragma unroll
  for (int t = 0; t < RT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      float s2 = 0.0f;
#pragma unroll
      for (int x = 0; x < ET; ++x) {
        const int e = (ew + x * (WAVES / RSPLIT)) * 16 + col;
        if (live[x] && e < a.E) s2 = fmaf(acc[x][t][r], acc[x][t][r], s2);
      }
#pragma unroll
      for (int off = 1; off < 16; off <<= 1) s2 += __shfl_xor(s2, off, 64);
      if (col == 0) sq[16 * (t0 + t) + 4 * grp + r][ew] = s2;
    }
  __syncthreads();
  if (tid < CR) {                         // a thread a row: one root for all its lanes
    float s2 = 0.0f;
#pragma unroll
    for (int y = 0; y < WAVES / RSPLIT; ++y) s2 += sq[tid][y];
    sq[tid][WAVES] = 1.0f / sqrtf(s2 / float(a.E) + a.eps);
  }
  __syncthreads();
#pragma unroll
  for (int t = 0; t < RT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * (t0 + t) + 4 * grp + r;
      if (i >= nr) continue;
      const float inv = sq[i][WAVES];
#pragma unroll
      for (int x = 0; x < ET; ++x) {
        const int e = (ew + x * (WAVES / RSPLIT)) * 16 + col;
        if (!live[x] || e >= a.E) continue;
        const float gt = gate[x][t][r];
        float y = acc[x][t][r] * inv;
        if (a.w) y *= ld_dyn(a.w, a.w_dtype, e);
        y *= gt * __builtin_amdgcn_rcpf(1.0f + exp2_f(-gt * kLog2e));
        const size_t at = size_t(r0 + i) * a.out_stride + head * a.E + e;
        if (a.out_dtype == SB_F32) ((float *)a.out)[at] = y;
        else ((bf16_t *)a.out)[at] = f32_to_bf16(y);
      }
    }
}

template <int DP, int CR, bool CHANNEL>
void launch_chunks(const ChunkArgs &a, int n_chunks, int n_seqs, hipStream_t s) {
  const dim3 grid(a.heads, n_chunks);
  if (a.E <= 64) chunk_local_kernel<DP, CR, 64, CHANNEL><<<grid, THREADS, 0, s>>>(a);
  else if (a.E <= 128) chunk_local_kernel<DP, CR, 128, CHANNEL><<<grid, THREADS, 0, s>>>(a);
  else chunk_local_kernel<DP, CR, 256, CHANNEL><<<grid, THREADS, 0, s>>>(a);
  chunk_carry_kernel<<<dim3(a.heads, n_seqs, (a.D * a.E + 255) / 256), 256, 0, s>>>(a, CR);
  if (a.E <= 64) chunk_from_kernel<DP, CR, 1, 2, CHANNEL><<<grid, THREADS, 0, s>>>(a);
  else if (a.E <= 128) chunk_from_kernel<DP, CR, 1, 1, CHANNEL><<<grid, THREADS, 0, s>>>(a);
  else chunk_from_kernel<DP, CR, 2, 1, CHANNEL><<<grid, THREADS, 0, s>>>(a);
}

template <bool CHANNEL>
void launch_by_dim(const ChunkArgs &a, int n_chunks, int n_seqs, hipStream_t s) {
  if (a.D <= 64) launch_chunks<64, 64, CHANNEL>(a, n_chunks, n_seqs, s);
  else if (a.D <= 128) launch_chunks<128, 64, CHANNEL>(a, n_chunks, n_seqs, s);
  else launch_chunks<256, 32, CHANNEL>(a, n_chunks, n_seqs, s);
}

__global__ void __launch_bounds__(256) angle_table_kernel(float2 *__restrict__ out, const int32_t *__restrict__ row_pos,
                                                          const float *__restrict__ inv_freq, int n_rows, int half) {
  const size_t idx = size_t(blockIdx.x) * 256 + threadIdx.x;
  if (idx >= size_t(n_rows) * half) return;
  const int row = int(idx / half), i = int(idx - size_t(row) * half);
  const float theta = float(row_pos[row]) * inv_freq[i];
  out[idx] = make_float2(cosf(theta), sinf(theta));
}

}  // namespace

// The rows of a chunk for heads of D key channels.
extern "C" int sb_decay_chunk_rows(int D) { return D <= 128 ? 64 : 32; }

// out f32 [n_rows, half, 2]: cosine and sine of row_pos[r] * inv_freq[i].
extern "C" int sb_angle_table(float *out, const int32_t *row_pos, const float *inv_freq, int n_rows, int half, void *stream) {
  SB_REQUIRE(out && row_pos && inv_freq, "sb_angle_table: null pointer");
  SB_REQUIRE(n_rows >= 0 && half > 0, "sb_angle_table: bad sizes rows=%d pairs=%d", n_rows, half);
  if (n_rows == 0) return SB_OK;
  const size_t n = size_t(n_rows) * half;
  angle_table_kernel<<<unsigned((n + 255) / 256), 256, 0, (hipStream_t)stream>>>((float2 *)out, row_pos, inv_freq, n_rows, half);
  return sb::check_launch("sb_angle_table");
}

// As sb_decay_scan, over n_chunks runs of at most sb_decay_chunk_rows(D) rows, sequence after sequence in row order,
// each sequence's runs full but its last.  angles f32 [n_rows, half, 2] or NULL; part f32 [n_chunks, heads, D, E] and,
// with log_decay, part_decay f32 [n_chunks, heads, D] are scratch.
extern "C" int sb_decay_chunks(void *out, int out_dtype, int out_stride, const float *q, const float *k, const float *v,
                               const float *g, int row_stride, const float *log_decay, int ld_stride, const float *decay,
                               const float *angles, int half, float q_scale, float k_scale, const void *w, int w_dtype,
                               float eps, float *state, const int32_t *cu_rows, const int32_t *slots, int n_seqs, int heads,
                               int D, int E, const int32_t *chunks, int n_chunks, int chunk_rows, float *part,
                               float *part_decay, int act_in, int plain, void *stream) {
  SB_REQUIRE(!plain || out_dtype == SB_F32, "sb_decay_chunks: what is read goes out in float32");
  SB_REQUIRE(out && q && k && v && (g || plain) && state && cu_rows && slots && chunks && part && (log_decay ? part_decay != nullptr : decay != nullptr),
             "sb_decay_chunks: null pointer");
  SB_REQUIRE(n_seqs >= 0 && n_chunks >= 0 && heads > 0 && D > 0 && E > 0 && sb::valid_dtype(out_dtype) && (!w || sb::valid_dtype(w_dtype)),
             "sb_decay_chunks: bad sizes heads=%d dim=%d vdim=%d", heads, D, E);
  SB_REQUIRE(!angles || (half > 0 && 2 * half <= D), "sb_decay_chunks: %d pairs do not fit a head of %d", half, D);
  SB_SUPPORT(D <= 256 && E <= 256, "sb_decay_chunks: a state of %d x %d a head is more than 256 x 256", D, E);
  SB_REQUIRE(chunk_rows == sb_decay_chunk_rows(D), "sb_decay_chunks: chunks of %d rows, heads of %d take %d", chunk_rows, D,
             sb_decay_chunk_rows(D));
  SB_SUPPORT(n_seqs <= 65535 && n_chunks <= 65535, "sb_decay_chunks: more than 65535 sequences or chunks");
  if (n_seqs == 0 || n_chunks == 0) return SB_OK;
  const auto aligned = [](const void *p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  const int vec4 = D % 4 == 0 && E % 4 == 0 && row_stride % 4 == 0 && aligned(q) && aligned(k) && aligned(v) && aligned(angles) &&
                   (!angles || half % 4 == 0);
  const ChunkArgs a{out, out_dtype, out_stride, q, k, v, g, row_stride, log_decay, ld_stride, decay, (const float2 *)angles,
                    angles ? half : 0, q_scale, k_scale, w, w_dtype, eps, state, cu_rows, slots, heads, D, E, chunks, part,
                    log_decay ? part_decay : nullptr, vec4, act_in, plain};
  if (log_decay) launch_by_dim<true>(a, n_chunks, n_seqs, (hipStream_t)stream);
  else launch_by_dim<false>(a, n_chunks, n_seqs, (hipStream_t)stream);
  return sb::check_launch("sb_decay_chunks");
}
