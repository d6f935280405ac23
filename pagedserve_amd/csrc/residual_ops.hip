// Steps on the float residual stream of layers whose sublayers add into a scratch row y that is
// folded into the stream with a factor, and what mixers that run side by side need.
#include <math.h>

#include "common.h"
#include "pagedserve_hip.h"

// One pass over the stream's rows, every piece optional:
//   h <- h + factor * column_scale * y + rows + bias;   zero <- 0 (may be y);
//   normed <- h / sqrt(mean(h^2) + eps) * gamma;   normed2 <- the same * gamma2
// (column_scale: a float per column, null for ones).  A block of 256 threads per token.
#define STREAM_HELD 8      // numbers of a row that a thread may hold
template <typename T>
__global__ __launch_bounds__(256) void stream_step_kernel(
    float* __restrict__ h, const float* y, float factor, const float* __restrict__ column_scale,
    const float* __restrict__ rows, const float* __restrict__ bias, const float* __restrict__ gamma, float eps,
    T* __restrict__ normed, const float* __restrict__ gamma2, T* __restrict__ normed2, float* zero, int width) {
  __shared__ float scratch[16];
  const int64_t t = blockIdx.x;
  float* row = h + t * width;
  float sum = 0.f;
  if (width <= 256 * STREAM_HELD) {
    // rows that a block holds in registers, with the scales asked for beside them: one trip to
    // memory and no second reading of the row
    float held[STREAM_HELD], scale[STREAM_HELD], scale2[STREAM_HELD];
#pragma unroll
    for (int i = 0; i < STREAM_HELD; ++i) {
      const int d = threadIdx.x + 256 * i;
      held[i] = scale[i] = scale2[i] = 0.f;
      if (d < width) {
        float v = row[d];
        if (gamma != nullptr) scale[i] = gamma[d];
        if (gamma2 != nullptr) scale2[i] = gamma2[d];
        if (y != nullptr) v = fmaf(column_scale ? factor * column_scale[d] : factor, y[t * width + d], v);
        if (rows != nullptr) v += rows[t * width + d];
        if (bias != nullptr) v += bias[d];
        held[i] = v;
      }
    }
#pragma unroll
    for (int i = 0; i < STREAM_HELD; ++i) {
      const int d = threadIdx.x + 256 * i;
      if (d < width) {
        if (y != nullptr || rows != nullptr || bias != nullptr) row[d] = held[i];
        if (zero != nullptr) zero[t * width + d] = 0.f;
      }
      sum = fmaf(held[i], held[i], sum);
    }
    if (gamma == nullptr) return;
    const float inv = 1.0f / sqrtf(block_sum(sum, scratch) / (float)width + eps);
#pragma unroll
    for (int i = 0; i < STREAM_HELD; ++i) {
      const int d = threadIdx.x + 256 * i;
      if (d < width) {
        normed[t * width + d] = from_float<T>(held[i] * inv * scale[i]);
        if (gamma2 != nullptr) normed2[t * width + d] = from_float<T>(held[i] * inv * scale2[i]);
      }
    }
    return;
  }
  for (int d = threadIdx.x; d < width; d += blockDim.x) {
    float v = row[d];
    if (y != nullptr) v = fmaf(column_scale ? factor * column_scale[d] : factor, y[t * width + d], v);
    if (rows != nullptr) v += rows[t * width + d];
    if (bias != nullptr) v += bias[d];
    if (y != nullptr || rows != nullptr || bias != nullptr) row[d] = v;
    if (zero != nullptr) zero[t * width + d] = 0.f;
    sum = fmaf(v, v, sum);
  }
  if (gamma == nullptr) return;
  const float inv = 1.0f / sqrtf(block_sum(sum, scratch) / (float)width + eps);
  // (each thread reads back what it wrote itself)
  for (int d = threadIdx.x; d < width; d += blockDim.x) {
    const float v = row[d] * inv;
    normed[t * width + d] = from_float<T>(v * gamma[d]);
    if (gamma2 != nullptr) normed2[t * width + d] = from_float<T>(v * gamma2[d]);
  }
}

// out[t, c] = unit(gu[t, c], gu[t, inner + c]) (common.h: GateForm), or act(gu[t, c]) * gu[t, inner + c]
// with ACT 1: gelu_tanh, 2: relu; times row_scale[t] where that is given
template <typename T, int ACT>
__global__ __launch_bounds__(256) void silu_gate_kernel(const float* __restrict__ gu, int64_t ld,
                                                        T* __restrict__ out, int64_t out_ld,
                                                        int inner, const GateForm form,
                                                        const float* __restrict__ row_scale) {
  const int64_t t = blockIdx.x;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= inner) return;
  const float g = gu[t * ld + c];
  const float u = gu[t * ld + inner + c];
  float v = ACT == 1 ? gelu_tanh_f(g) * u : (ACT == 2 ? fmaxf(g, 0.f) * u : gated_unit(g, u, form));
  if (row_scale != nullptr) v *= row_scale[t];
  out[t * out_ld + c] = from_float<T>(v);
}

// p[t, c] <- silu(p[t, c]) for columns first .. first + count - 1 of rows ld floats apart
__global__ __launch_bounds__(256) void silu_columns_kernel(float* __restrict__ p, int64_t ld, int first,
                                                           int count) {
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= count) return;
  float* at = p + (int64_t)blockIdx.x * ld + first + c;
  const float v = *at;
  *at = v / (1.0f + expf(-v));
}

// y <- y + share * (a / rms(a) * wa + b / rms(b) * wb);  a <- 0;  b <- 0.   A block per token.
__global__ __launch_bounds__(256) void pair_norm_mix_kernel(
    float* __restrict__ a, float* __restrict__ b, const float* __restrict__ wa,
    const float* __restrict__ wb, float eps, float share, float* __restrict__ y, int width) {
  __shared__ float scratch_a[16], scratch_b[16];
  const int64_t t = blockIdx.x;
  float* ra = a + t * width;
  float* rb = b + t * width;
  float sa = 0.f, sb = 0.f;
  for (int d = threadIdx.x; d < width; d += blockDim.x) {
    sa = fmaf(ra[d], ra[d], sa);
    sb = fmaf(rb[d], rb[d], sb);
  }
  const float ia = 1.0f / sqrtf(block_sum(sa, scratch_a) / (float)width + eps);
  const float ib = 1.0f / sqrtf(block_sum(sb, scratch_b) / (float)width + eps);
  for (int d = threadIdx.x; d < width; d += blockDim.x) {
    const float va = ra[d] * ia * wa[d];
    const float vb = rb[d] * ib * wb[d];
    y[t * width + d] += share * (va + vb);
    ra[d] = 0.f;
    rb[d] = 0.f;
  }
}

extern "C" int ps_stream_step(float* h, const float* y, float factor, const float* column_scale,
                              const float* rows, const float* bias, const float* gamma, float eps,
                              void* normed, const float* gamma2, void* normed2, float* zero, int tokens,
                              int width, int out_dtype, void* stream) {
  PS_REQUIRE(tokens >= 0 && width > 0, "ps_stream_step: bad sizes");
  PS_REQUIRE(gamma == nullptr || (normed != nullptr && eps > 0.f),
             "ps_stream_step: a norm needs an output and a positive eps");
  PS_REQUIRE(gamma2 == nullptr || (gamma != nullptr && normed2 != nullptr),
             "ps_stream_step: a second scale goes with the first and needs an output");
  PS_REQUIRE(out_dtype == PS_F32 || out_dtype == PS_BF16, "ps_stream_step: unknown dtype %d", out_dtype);
  if (tokens == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  if (out_dtype == PS_F32)
    hipLaunchKernelGGL(stream_step_kernel<float>, dim3(tokens), dim3(256), 0, s, h, y, factor,
                       column_scale, rows, bias, gamma, eps, (float*)normed, gamma2, (float*)normed2, zero, width);
  else
    hipLaunchKernelGGL(stream_step_kernel<bf16_t>, dim3(tokens), dim3(256), 0, s, h, y, factor,
                       column_scale, rows, bias, gamma, eps, (bf16_t*)normed, gamma2, (bf16_t*)normed2, zero, width);
  PS_CHECK_LAUNCH("ps_stream_step");
  return 0;
}

extern "C" int ps_silu_gate(const float* gu, int64_t ld, void* out, int64_t out_ld, int tokens,
                            int inner, int activation, float limit, float slope, float shift,
                            const float* row_scale, int dtype, void* stream) {
  PS_REQUIRE(tokens >= 0 && inner > 0 && ld >= 2 * (int64_t)inner && out_ld >= inner,
             "ps_silu_gate: bad sizes");
  PS_REQUIRE(dtype == PS_F32 || dtype == PS_BF16, "ps_silu_gate: unknown dtype %d", dtype);
  if (tokens == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const dim3 grid(tokens, (inner + 255) / 256);
  PS_REQUIRE(activation >= 0 && activation <= 2, "ps_silu_gate: activation %d (0: silu, 1: gelu_tanh, 2: relu)", activation);
  PS_REQUIRE(limit > 0.f, "ps_silu_gate: the limit must be positive");
  const GateForm form = {limit, slope, shift};
#define PS_LAUNCH_SG(T, ACT) \
  hipLaunchKernelGGL((silu_gate_kernel<T, ACT>), grid, dim3(256), 0, s, gu, ld, (T*)out, out_ld, inner, form, row_scale)
#define PS_LAUNCH_SG_T(T)                          \
  do {                                             \
    if (activation == 1) PS_LAUNCH_SG(T, 1);       \
    else if (activation == 2) PS_LAUNCH_SG(T, 2);  \
    else PS_LAUNCH_SG(T, 0);                       \
  } while (0)
  if (dtype == PS_F32) PS_LAUNCH_SG_T(float);
  else PS_LAUNCH_SG_T(bf16_t);
#undef PS_LAUNCH_SG_T
#undef PS_LAUNCH_SG
  PS_CHECK_LAUNCH("ps_silu_gate");
  return 0;
}

extern "C" int ps_silu_columns(float* p, int64_t ld, int first, int count, int tokens, void* stream) {
  PS_REQUIRE(tokens >= 0 && first >= 0 && count > 0 && ld >= first + count, "ps_silu_columns: bad sizes");
  if (tokens == 0) return 0;
  hipLaunchKernelGGL(silu_columns_kernel, dim3(tokens, (count + 255) / 256), dim3(256), 0,
                     (hipStream_t)stream, p, ld, first, count);
  PS_CHECK_LAUNCH("ps_silu_columns");
  return 0;
}

extern "C" int ps_pair_norm_mix(float* a, float* b, const float* wa, const float* wb, float eps,
                                float share, float* y, int tokens, int width, void* stream) {
  PS_REQUIRE(tokens >= 0 && width > 0 && eps > 0.f, "ps_pair_norm_mix: bad sizes");
  if (tokens == 0) return 0;
  hipLaunchKernelGGL(pair_norm_mix_kernel, dim3(tokens), dim3(256), 0, (hipStream_t)stream, a, b, wa,
                     wb, eps, share, y, width);
  PS_CHECK_LAUNCH("ps_pair_norm_mix");
  return 0;
}

// Sublayers between two layer norms, with a gate on their result.  Per token, one pass:
//   h <- h + LN(sigmoid(gate + gate_bias) * y; gamma, beta);   y <- 0
//   normed <- LN(h; gamma2, beta2)
// with LN(x) = (x - mean) / sqrt(mean((x - mean)^2) + eps) * gamma + beta; either half is optional.  A
// block holds its row in registers, HELD numbers to a thread.
template <typename T, int HELD>
__global__ __launch_bounds__(1024) void gated_norm_step_kernel(
    float* __restrict__ h, float* __restrict__ y, const float* __restrict__ gate, int64_t gate_ld,
    const float* __restrict__ gate_bias, const float* __restrict__ gamma, const float* __restrict__ beta,
    const float* __restrict__ gamma2, const float* __restrict__ beta2, float eps, T* __restrict__ normed,
    int width) {
  __shared__ float scratch[16];
  const int64_t t = blockIdx.x;
  float* row = h + t * width;
  float x[HELD], v[HELD], scale[HELD], shift[HELD], scale2[HELD], shift2[HELD];
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < HELD; ++i) {
    const int d = threadIdx.x + blockDim.x * i;
    x[i] = v[i] = scale[i] = shift[i] = scale2[i] = shift2[i] = 0.f;
    if (d < width) {
      x[i] = row[d];
      if (gamma2 != nullptr) {
        scale2[i] = gamma2[d];
        shift2[i] = beta2[d];
      }
      if (y != nullptr) {
        scale[i] = gamma[d];
        shift[i] = beta[d];
        v[i] = y[t * width + d] / (1.0f + expf(-(gate[t * gate_ld + d] + gate_bias[d])));
        y[t * width + d] = 0.f;
      }
    }
    sum += v[i];
  }
  if (y != nullptr) {
    const float mean = block_sum(sum, scratch) / (float)width;
    float squares = 0.f;
#pragma unroll
    for (int i = 0; i < HELD; ++i) {
      const int d = threadIdx.x + blockDim.x * i;
      v[i] = d < width ? v[i] - mean : 0.f;
      squares = fmaf(v[i], v[i], squares);
    }
    const float inv = 1.0f / sqrtf(block_sum(squares, scratch) / (float)width + eps);
#pragma unroll
    for (int i = 0; i < HELD; ++i) {
      const int d = threadIdx.x + blockDim.x * i;
      x[i] += fmaf(v[i] * inv, scale[i], shift[i]);
      if (d < width) row[d] = x[i];
    }
  }
  if (gamma2 == nullptr) return;
  sum = 0.f;
#pragma unroll
  for (int i = 0; i < HELD; ++i) sum += x[i];
  const float mean = block_sum(sum, scratch) / (float)width;
  float squares = 0.f;
#pragma unroll
  for (int i = 0; i < HELD; ++i) {
    const int d = threadIdx.x + blockDim.x * i;
    x[i] = d < width ? x[i] - mean : 0.f;
    squares = fmaf(x[i], x[i], squares);
  }
  const float inv = 1.0f / sqrtf(block_sum(squares, scratch) / (float)width + eps);
#pragma unroll
  for (int i = 0; i < HELD; ++i) {
    const int d = threadIdx.x + blockDim.x * i;
    if (d < width) normed[t * width + d] = from_float<T>(fmaf(x[i] * inv, scale2[i], shift2[i]));
  }
}

extern "C" int ps_gated_norm_step(float* h, float* y, const float* gate, int64_t gate_ld,
                                  const float* gate_bias, const float* gamma, const float* beta,
                                  const float* gamma2, const float* beta2, float eps, void* normed,
                                  int tokens, int width, int out_dtype, void* stream) {
  PS_REQUIRE(tokens >= 0 && width > 0 && width <= 16384 && eps > 0.f,
             "ps_gated_norm_step: bad sizes (width %d, at most 16384)", width);
  PS_REQUIRE(y == nullptr || (gate != nullptr && gate_bias != nullptr && gamma != nullptr && beta != nullptr && gate_ld >= width),
             "ps_gated_norm_step: a result needs its gate and its norm");
  PS_REQUIRE(gamma2 == nullptr || (beta2 != nullptr && normed != nullptr),
             "ps_gated_norm_step: a second norm needs its shift and an output");
  PS_REQUIRE(out_dtype == PS_F32 || out_dtype == PS_BF16, "ps_gated_norm_step: unknown dtype %d", out_dtype);
  if (tokens == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  // few rows wait for their trips to memory: a thread per column as far as a block has them; many
  // rows fill the chip with blocks of four waves
  int threads = width >= 1024 ? 1024 : (width + 63) / 64 * 64;
  if (tokens > 256 && threads > 256 && width <= 256 * 16) threads = 256;
  const int held = (width + threads - 1) / threads;
#define PS_LAUNCH_GNS(T, HELD)                                                                          \
  hipLaunchKernelGGL((gated_norm_step_kernel<T, HELD>), dim3(tokens), dim3(threads), 0, s, h, y, gate,  \
                     gate_ld, gate_bias, gamma, beta, gamma2, beta2, eps, (T*)normed, width)
#define PS_LAUNCH_GNS_T(T)                       \
  do {                                           \
    if (held <= 1) PS_LAUNCH_GNS(T, 1);          \
    else if (held <= 2) PS_LAUNCH_GNS(T, 2);     \
    else if (held <= 4) PS_LAUNCH_GNS(T, 4);     \
    else if (held <= 8) PS_LAUNCH_GNS(T, 8);     \
    else PS_LAUNCH_GNS(T, 16);                   \
  } while (0)
  if (out_dtype == PS_F32) PS_LAUNCH_GNS_T(float);
  else PS_LAUNCH_GNS_T(bf16_t);
#undef PS_LAUNCH_GNS_T
#undef PS_LAUNCH_GNS
  PS_CHECK_LAUNCH("ps_gated_norm_step");
  return 0;
}
