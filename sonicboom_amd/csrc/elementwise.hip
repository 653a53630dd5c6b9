// Gated product, residual add, type conversion.
//
// act(g) * u with the gate's activation (SiLU with the full-precision expf, or the tanh form
// of GELU: gate_act in common.h), u the up projection
// (/root/reference/core/src/nn/activation.cpp:27-50, /root/reference/core/src/model/emit.cpp:364-374).
#include "common.h"

namespace {

template <typename TO, typename TI>
__global__ void gate_mul_kernel(TO *__restrict__ out, const TI *__restrict__ gu, int width,
                                size_t total, int gate) {
  const size_t idx = size_t(blockIdx.x) * blockDim.x + threadIdx.x;
  if (idx >= total) return;
  const size_t row = idx / width;
  const int col = int(idx - row * width);
  const TI *g_row = gu + row * size_t(2 * width);
  const float g = ld_f(g_row, col);
  const float u = ld_f(g_row, size_t(width) + col);
  st_f(out, idx, gate_act(g, gate) * u);
}

template <typename TI>
__global__ void add_into_kernel(float *__restrict__ resid, const TI *__restrict__ y, size_t n) {
  const size_t idx = size_t(blockIdx.x) * blockDim.x + threadIdx.x;
  if (idx < n) resid[idx] = ld_f(y, idx) + resid[idx];
}

template <typename TO, typename TI>
__global__ void cast_kernel(TO *__restrict__ dst, const TI *__restrict__ src, size_t n) {
  const size_t idx = size_t(blockIdx.x) * blockDim.x + threadIdx.x;
  if (idx < n) st_f(dst, idx, ld_f(src, idx));
}

inline unsigned blocks_for(size_t n, int threads) { return unsigned((n + threads - 1) / threads); }

}  // namespace

extern "C" int sb_gate_mul(void *out, int out_dtype, const void *gu, int gu_dtype, int n_rows,
                           int width, int gate, void *stream) {
  SB_REQUIRE(out && gu, "sb_gate_mul: null pointer");
  SB_REQUIRE(n_rows >= 0 && width > 0, "sb_gate_mul: bad sizes rows=%d width=%d", n_rows, width);
  SB_REQUIRE(sb::valid_dtype(out_dtype) && sb::valid_dtype(gu_dtype), "sb_gate_mul: unknown dtype");
  SB_SUPPORT(gate >= SB_GATE_SILU && gate <= SB_GATE_RELU, "sb_gate_mul: unknown gate activation %d", gate);
  const size_t total = size_t(n_rows) * width;
  if (total == 0) return SB_OK;
  hipStream_t s = (hipStream_t)stream;
  const unsigned nb = blocks_for(total, 256);
#define SB_GO(TO, TI) gate_mul_kernel<TO, TI><<<nb, 256, 0, s>>>((TO *)out, (const TI *)gu, width, total, gate)
  if (out_dtype == SB_F32 && gu_dtype == SB_F32) SB_GO(float, float);
  else if (out_dtype == SB_BF16 && gu_dtype == SB_F32) SB_GO(bf16_t, float);
  else if (out_dtype == SB_BF16 && gu_dtype == SB_BF16) SB_GO(bf16_t, bf16_t);
  else SB_GO(float, bf16_t);
#undef SB_GO
  return sb::check_launch("sb_gate_mul");
}

extern "C" int sb_silu_mul(void *out, int out_dtype, const void *gu, int gu_dtype, int n_rows,
                           int width, void *stream) {
  return sb_gate_mul(out, out_dtype, gu, gu_dtype, n_rows, width, SB_GATE_SILU, stream);
}

extern "C" int sb_add_into(float *resid, const void *y, int y_dtype, size_t n, void *stream) {
  SB_REQUIRE(resid && y, "sb_add_into: null pointer");
  SB_REQUIRE(sb::valid_dtype(y_dtype), "sb_add_into: unknown dtype");
  if (n == 0) return SB_OK;
  hipStream_t s = (hipStream_t)stream;
  const unsigned nb = blocks_for(n, 256);
  if (y_dtype == SB_F32) add_into_kernel<float><<<nb, 256, 0, s>>>(resid, (const float *)y, n);
  else add_into_kernel<bf16_t><<<nb, 256, 0, s>>>(resid, (const bf16_t *)y, n);
  return sb::check_launch("sb_add_into");
}

extern "C" int sb_cast(void *dst, int dst_dtype, const void *src, int src_dtype, size_t n,
                       void *stream) {
  SB_REQUIRE(dst && src, "sb_cast: null pointer");
  SB_REQUIRE(sb::valid_dtype(dst_dtype) && sb::valid_dtype(src_dtype), "sb_cast: unknown dtype");
  if (n == 0) return SB_OK;
  hipStream_t s = (hipStream_t)stream;
  const unsigned nb = blocks_for(n, 256);
#define SB_GO(TO, TI) cast_kernel<TO, TI><<<nb, 256, 0, s>>>((TO *)dst, (const TI *)src, n)
  if (dst_dtype == SB_F32 && src_dtype == SB_F32) SB_GO(float, float);
  else if (dst_dtype == SB_BF16 && src_dtype == SB_F32) SB_GO(bf16_t, float);
  else if (dst_dtype == SB_BF16 && src_dtype == SB_BF16) SB_GO(bf16_t, bf16_t);
  else SB_GO(float, bf16_t);
#undef SB_GO
  return sb::check_launch("sb_cast");
}

// ---- a scaled residual add, and activations of an ungated feed-forward ------------------------
namespace {

template <typename TI>
__global__ void add_scaled_kernel(float *__restrict__ resid, const TI *__restrict__ y, float scale, size_t n) {
  const size_t idx = size_t(blockIdx.x) * blockDim.x + threadIdx.x;
  if (idx < n) resid[idx] = ld_f(y, idx) * scale + resid[idx];
}

__device__ __forceinline__ float softplus_f(float a) { return a > 20.0f ? a : log1pf(expf(a)); }

// xIELU with the two numbers (p, q) of a layer: for z > 0 softplus(p) z^2 + z/2, else
// (1/2 + softplus(q)) (exp(z) - 1 - z) + z/2.
__device__ __forceinline__ float activate_one(float z, int kind, float ap, float an) {
  if (kind == SB_ACT_XIELU) return z > 0.0f ? ap * z * z + 0.5f * z : an * (expm1f(z) - z) + 0.5f * z;
  if (kind == SB_ACT_GELU_ERF) return 0.5f * z * (1.0f + erff(z * 0.70710678118654752440f));      // z Phi(z) by the error function
  if (kind == SB_ACT_RELU_SQ) { const float r = fmaxf(z, 0.0f); return r * r; }
  return gate_act(z, kind == SB_ACT_GELU_TANH ? SB_GATE_GELU_TANH : SB_GATE_SILU);
}

// A thread takes four neighbouring elements (n4 groups of four, then the tail one by one).
template <typename TO, typename TI>
__global__ void activate_kernel(TO *__restrict__ out, const TI *__restrict__ in, size_t n, size_t n4, int kind,
                                const void *__restrict__ params, int params_dtype) {
  const size_t idx = size_t(blockIdx.x) * blockDim.x + threadIdx.x;
  float ap = 0.0f, an = 0.0f;
  if (kind == SB_ACT_XIELU) {
    ap = softplus_f(ld_dyn(params, params_dtype, 0));
    an = 0.5f + softplus_f(ld_dyn(params, params_dtype, 1));
  }
  if (idx < n4) {
    float z[4];
    if constexpr (sizeof(TI) == 4) {
      const float4 v = reinterpret_cast<const float4 *>(in)[idx];
      z[0] = v.x; z[1] = v.y; z[2] = v.z; z[3] = v.w;
    } else {
      const uint2 v = reinterpret_cast<const uint2 *>(in)[idx];
      z[0] = bf16_to_f32(bf16_t(v.x & 0xffffu)); z[1] = bf16_to_f32(bf16_t(v.x >> 16));
      z[2] = bf16_to_f32(bf16_t(v.y & 0xffffu)); z[3] = bf16_to_f32(bf16_t(v.y >> 16));
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) z[e] = activate_one(z[e], kind, ap, an);
    if constexpr (sizeof(TO) == 4) {
      reinterpret_cast<float4 *>(out)[idx] = make_float4(z[0], z[1], z[2], z[3]);
    } else {
      reinterpret_cast<uint2 *>(out)[idx] = make_uint2(uint32_t(f32_to_bf16(z[0])) | uint32_t(f32_to_bf16(z[1])) << 16,
                                                       uint32_t(f32_to_bf16(z[2])) | uint32_t(f32_to_bf16(z[3])) << 16);
    }
  } else {
    const size_t i = 4 * n4 + (idx - n4);
    if (i < n) st_f(out, i, activate_one(ld_f(in, i), kind, ap, an));
  }
}

// out = act(the sum of K slices + bias), numbers of a row of `width` in fours: every slice asked for before any is added.
template <typename TO>
__global__ void __launch_bounds__(256)
activate_slices_kernel(TO *__restrict__ out, const float *__restrict__ in, int n_slices, size_t slice_stride, const float *__restrict__ bias,
                       int width, size_t n4, int kind, const void *__restrict__ params, int params_dtype) {
  const size_t idx = size_t(blockIdx.x) * 256 + threadIdx.x;
  if (idx >= n4) return;
  float ap = 0.0f, an = 0.0f;
  if (kind == SB_ACT_XIELU) {
    ap = softplus_f(ld_dyn(params, params_dtype, 0));
    an = 0.5f + softplus_f(ld_dyn(params, params_dtype, 1));
  }
  float4 part[kSliceLoads];
#pragma unroll
  for (int s = 0; s < kSliceLoads; ++s) part[s] = *reinterpret_cast<const float4 *>(in + min(s, n_slices - 1) * slice_stride + 4 * idx);
  float z[4] = {part[0].x, part[0].y, part[0].z, part[0].w};
#pragma unroll
  for (int s = 1; s < kSliceLoads; ++s)
    if (s < n_slices) { z[0] += part[s].x; z[1] += part[s].y; z[2] += part[s].z; z[3] += part[s].w; }
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    if (bias) z[e] += bias[(4 * idx) % width + e];
    z[e] = activate_one(z[e], kind, ap, an);
  }
  if constexpr (sizeof(TO) == 4)
    reinterpret_cast<float4 *>(out)[idx] = make_float4(z[0], z[1], z[2], z[3]);
  else
    reinterpret_cast<uint2 *>(out)[idx] = make_uint2(uint32_t(f32_to_bf16(z[0])) | uint32_t(f32_to_bf16(z[1])) << 16,
                                                     uint32_t(f32_to_bf16(z[2])) | uint32_t(f32_to_bf16(z[3])) << 16);
}

}  // namespace

// in f32 [n_slices][n_rows * width], width a multiple of 4, up to 8 slices; bias f32 [width] or NULL.
extern "C" int sb_activate_slices(void *out, int out_dtype, const float *in, int n_slices, const float *bias, int n_rows, int width, int kind,
                                  const void *params, int params_dtype, void *stream) {
  SB_REQUIRE(out && in && n_rows >= 0 && width > 0 && n_slices > 0, "sb_activate_slices: bad sizes rows=%d width=%d slices=%d", n_rows, width,
             n_slices);
  SB_REQUIRE(sb::valid_dtype(out_dtype) && kind >= SB_ACT_SILU && kind <= SB_ACT_RELU_SQ, "sb_activate_slices: unknown type or activation");
  SB_REQUIRE(kind != SB_ACT_XIELU || (params && sb::valid_dtype(params_dtype)), "sb_activate_slices: xIELU takes two numbers");
  SB_SUPPORT(width % 4 == 0 && n_slices <= kSliceLoads && ((reinterpret_cast<uintptr_t>(in) | reinterpret_cast<uintptr_t>(out)) & 15) == 0,
             "sb_activate_slices: rows of %d in %d slices", width, n_slices);
  const size_t n4 = size_t(n_rows) * width / 4;
  if (n4 == 0) return SB_OK;
  hipStream_t s = (hipStream_t)stream;
  const unsigned nb = blocks_for(n4, 256);
  if (out_dtype == SB_F32)
    activate_slices_kernel<float><<<nb, 256, 0, s>>>((float *)out, in, n_slices, 4 * n4, bias, width, n4, kind, params, params_dtype);
  else activate_slices_kernel<bf16_t><<<nb, 256, 0, s>>>((bf16_t *)out, in, n_slices, 4 * n4, bias, width, n4, kind, params, params_dtype);
  return sb::check_launch("sb_activate_slices");
}

extern "C" int sb_add_scaled(float *resid, const void *y, int y_dtype, float scale, size_t n, void *stream) {
  SB_REQUIRE(resid && y, "sb_add_scaled: null pointer");
  SB_REQUIRE(sb::valid_dtype(y_dtype), "sb_add_scaled: unknown dtype");
  if (n == 0) return SB_OK;
  hipStream_t s = (hipStream_t)stream;
  const unsigned nb = blocks_for(n, 256);
  if (y_dtype == SB_F32) add_scaled_kernel<float><<<nb, 256, 0, s>>>(resid, (const float *)y, scale, n);
  else add_scaled_kernel<bf16_t><<<nb, 256, 0, s>>>(resid, (const bf16_t *)y, scale, n);
  return sb::check_launch("sb_add_scaled");
}

extern "C" int sb_activate(void *out, int out_dtype, const void *in, int in_dtype, size_t n, int kind,
                           const void *params, int params_dtype, void *stream) {
  SB_REQUIRE(out && in, "sb_activate: null pointer");
  SB_REQUIRE(sb::valid_dtype(out_dtype) && sb::valid_dtype(in_dtype), "sb_activate: unknown dtype");
  SB_SUPPORT(kind == SB_ACT_SILU || kind == SB_ACT_GELU_TANH || kind == SB_ACT_XIELU || kind == SB_ACT_GELU_ERF || kind == SB_ACT_RELU_SQ,
             "sb_activate: unknown activation %d", kind);
  SB_REQUIRE(kind != SB_ACT_XIELU || (params && sb::valid_dtype(params_dtype)),
             "sb_activate: xIELU needs its two numbers");
  if (n == 0) return SB_OK;
  hipStream_t s = (hipStream_t)stream;
  // groups of four where both buffers start on 16 bytes (every tensor of the engine does)
  const bool vec = ((reinterpret_cast<uintptr_t>(out) | reinterpret_cast<uintptr_t>(in)) & 15) == 0;
  const size_t n4 = vec ? n / 4 : 0;
  const unsigned nb = blocks_for(n4 + (n - 4 * n4), 256);
#define SB_GO(TO, TI) activate_kernel<TO, TI><<<nb, 256, 0, s>>>((TO *)out, (const TI *)in, n, n4, kind, params, params_dtype)
  if (out_dtype == SB_F32 && in_dtype == SB_F32) SB_GO(float, float);
  else if (out_dtype == SB_BF16 && in_dtype == SB_F32) SB_GO(bf16_t, float);
  else if (out_dtype == SB_BF16 && in_dtype == SB_BF16) SB_GO(bf16_t, bf16_t);
  else SB_GO(float, bf16_t);
#undef SB_GO
  return sb::check_launch("sb_activate");
}

// ---- a sigmoid gate on finished rows, and a cap on logits ------------------------------------------------
namespace {

// x[t, i] *= sigmoid(gate[t * gate_stride + i]): x in the activation type, the gate's rows float32
// (a part of a wider product's rows).  The sigmoid in float32 with the full-precision exponential.
template <typename TX>
__global__ void sigmoid_mul_kernel(TX *__restrict__ x, const float *__restrict__ gate, int gate_stride, int width, size_t n) {
  const size_t idx = size_t(blockIdx.x) * blockDim.x + threadIdx.x;
  if (idx >= n) return;
  const size_t t = idx / width, i = idx - t * width;
  const float g = gate[t * gate_stride + i];
  st_f(x, idx, ld_f(x, idx) * (1.0f / (1.0f + expf(-g))));
}

__global__ void softcap_kernel(float *__restrict__ x, float cap, size_t n) {
  const size_t idx = size_t(blockIdx.x) * blockDim.x + threadIdx.x;
  if (idx < n) x[idx] = cap * tanhf(x[idx] / cap);
}

}  // namespace

extern "C" int sb_sigmoid_mul(void *x, int x_dtype, const float *gate, int gate_stride, int n_rows, int width, void *stream) {
  SB_REQUIRE(x && gate, "sb_sigmoid_mul: null pointer");
  SB_REQUIRE(n_rows >= 0 && width > 0 && gate_stride >= width && sb::valid_dtype(x_dtype),
             "sb_sigmoid_mul: bad sizes rows=%d width=%d stride=%d", n_rows, width, gate_stride);
  const size_t n = size_t(n_rows) * width;
  if (n == 0) return SB_OK;
  hipStream_t s = (hipStream_t)stream;
  const unsigned nb = blocks_for(n, 256);
  if (x_dtype == SB_F32) sigmoid_mul_kernel<float><<<nb, 256, 0, s>>>((float *)x, gate, gate_stride, width, n);
  else sigmoid_mul_kernel<bf16_t><<<nb, 256, 0, s>>>((bf16_t *)x, gate, gate_stride, width, n);
  return sb::check_launch("sb_sigmoid_mul");
}

// x <- cap tanh(x / cap), element by element, float32 in place (logits).
extern "C" int sb_softcap(float *x, float cap, size_t n, void *stream) {
  SB_REQUIRE(x, "sb_softcap: null pointer");
  SB_REQUIRE(cap > 0.0f, "sb_softcap: the cap must be positive");
  if (n == 0) return SB_OK;
  softcap_kernel<<<blocks_for(n, 256), 256, 0, (hipStream_t)stream>>>(x, cap, n);
  return sb::check_launch("sb_softcap");
}

// ---- measurement: how fast can this GPU stream memory? ---------------------------------------
namespace {
__global__ void __launch_bounds__(256)
read_probe_kernel(uint32_t *__restrict__ sink, const uint4 *__restrict__ src, size_t n_vec) {
  const size_t stride = size_t(gridDim.x) * blockDim.x;
  size_t i = size_t(blockIdx.x) * blockDim.x + threadIdx.x;
  uint32_t acc = 0;
  for (; i + 3 * stride < n_vec; i += 4 * stride) {
    const uint4 a = src[i], b = src[i + stride], c = src[i + 2 * stride], d = src[i + 3 * stride];
    acc ^= a.x ^ a.y ^ a.z ^ a.w ^ b.x ^ b.y ^ b.z ^ b.w ^ c.x ^ c.y ^ c.z ^ c.w ^ d.x ^ d.y ^ d.z ^ d.w;
  }
  for (; i < n_vec; i += stride) {
    const uint4 a = src[i];
    acc ^= a.x ^ a.y ^ a.z ^ a.w;
  }
  if (acc == 0x9e3779b9u) sink[0] = acc;   // keeps the loads alive; practically never taken
}
}  // namespace

// Reads `bytes` (a multiple of 16) from src once with `blocks` blocks of 256 threads, 16 bytes
// per load, four loads in flight per thread.  For timing the memory system; writes nothing
// worth reading.
extern "C" int sb_read_probe(void *sink, const void *src, size_t bytes, int blocks, void *stream) {
  SB_REQUIRE(sink && src && blocks > 0, "sb_read_probe: bad arguments");
  read_probe_kernel<<<blocks, 256, 0, (hipStream_t)stream>>>((uint32_t *)sink, (const uint4 *)src, bytes / 16);
  return sb::check_launch("sb_read_probe");
}

// ---- a multiplier on float32 values in place (the logits of a head that has one) ---------------
namespace {
__global__ void scale_kernel(float *__restrict__ x, float scale, size_t n) {
  const size_t i = size_t(blockIdx.x) * blockDim.x + threadIdx.x;
  if (i < n) x[i] = x[i] * scale;
}
}  // namespace

extern "C" int sb_scale(float *x, float scale, size_t n, void *stream) {
  SB_REQUIRE(x || n == 0, "sb_scale: null pointer");
  if (n == 0) return SB_OK;
  scale_kernel<<<unsigned((n + 255) / 256), 256, 0, (hipStream_t)stream>>>(x, scale, n);
  return sb::check_launch("sb_scale");
}
