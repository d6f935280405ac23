// The decayed rule of matrix_state.hip for long portions, on the matrix cores (bfloat16 engine).
//
// With one decay per head and token the recurrence is linear in the state, and a run of tokens can be
// worked out at once.  The items of a step are cut into pieces of up to SC_TOKENS tokens.  Within a piece let
// L_t be the sum of the logarithms of the decays up to and including token t, L the piece's whole sum, S0
// the state at its start:
//
//   what the piece adds   E = sum_t e^(L - L_t) w_t k_t v_t^T                    (all pieces side by side)
//   its start             S0 of the next piece = e^L S0 + E                      (piece after piece, per number)
//   its outputs           o_t = e^(L_t) S0^T q_t + sum_(s <= t) e^(L_t - L_s) w_s (q_t . k_s) v_s    (side by side)
//
// Queries, keys and values are what projections and convolutions left and enter the products as
// bfloat16; everything that carries decays, weights or the state is float and enters as two
// bfloat16 parts, x = hi + lo, so that a product keeps 16 bits of it.  Sums are float.
#include <math.h>

#include "common.h"
#include "matrix_state.h"
#include "pagedserve_hip.h"

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float f32x4;

#define SC_TOKENS 64
#define SC_ROW (SC_TOKENS + 8)     // bf16 per row of an operand whose rows run along the tokens

struct ChunkArgs {
  StateStep s;
  const int* piece_cu;      // token ranges of the pieces, empty behind the last one
  const int* item_first;    // the first piece of each item
  float* records;           // [pieces][heads][columns][key_dim]: what a piece adds, then its start
  float* totals;            // [pieces][heads]: the sum of its logarithms
};

__device__ inline bf16x8 as_operand(const uint4& v) { return *reinterpret_cast<const bf16x8*>(&v); }

// s_log[t] = L_t, s_take[t] = w_t of the piece's tokens (wave 0; zero weight and no decay behind the last token).
__device__ inline void piece_decays(const StateStep& p, int head, int t0, int count, float* s_log, float* s_take) {
  if (threadIdx.x < 64) {
    const int lane = threadIdx.x;
    const int64_t at = (int64_t)(t0 + (lane < count ? lane : count - 1)) * p.heads + head;
    float sum = lane < count ? p.decay[at] : 0.f;
    const float w = lane < count ? p.take[at] : 0.f;
#pragma unroll
    for (int step = 1; step < 64; step <<= 1) {
      const float before = __shfl_up(sum, step, 64);
      if (lane >= step) sum += before;
    }
    s_log[lane] = sum;
    s_take[lane] = w;
  }
}

// x = row[first .. first + 3].  VEC: rows begin at multiples of 16 bytes and their sizes are multiples of 4;
// beyond a row's end the loads come from its last numbers (no branch stands between the loads of a
// thread: they all leave together, and the caller masks).
template <bool VEC>
__device__ inline void piece_four(const float* row, int first, int size, float* x) {
  if (VEC) {
    *reinterpret_cast<float4*>(x) = *reinterpret_cast<const float4*>(row + (first + 4 <= size ? first : size - 4));
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i) x[i] = row[first + i < size ? first + i : size - 1];
  }
}

// Rows of the piece's tokens into LDS with the tokens side by side: put(d, tt, x0, x1) gets columns first + d,
// d < rows, of tokens tt and tt + 1 (what lies behind the last token or column is whatever a clamped address
// holds: the caller masks).  The block's threads: 16 lanes share 64 columns of a token, a wave takes 8
// tokens at a time.
template <bool VEC, typename Put>
__device__ inline void stage_transposed(const float* base, int64_t ld, int count, int first, int size, int rows,
                                        Put put) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int tt = wave * 16 + (lane >> 4) * 2;
  for (int d0 = 0; d0 < rows; d0 += 64) {
    const int d = d0 + (lane & 15) * 4;
    float x[2][2][4];
#pragma unroll
    for (int turn = 0; turn < 2; ++turn)
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const int t = tt + turn * 8 + j;
        piece_four<VEC>(base + (int64_t)(t < count ? t : count - 1) * ld, first + d, size, x[turn][j]);
      }
#pragma unroll
    for (int turn = 0; turn < 2; ++turn)
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (d + i < rows) put(d + i, tt + turn * 8, x[turn][0][i], x[turn][1][i]);
  }
}

// Where key dimension d (of a run of 32) stands among the places of the products over the key dimensions: a
// lane's eight places hold dimensions 4 g .. 4 g + 3 and 16 + 4 g .. 16 + 4 g + 3, so that its two loads of 16
// bytes lie side by side with its neighbours'.
__device__ inline int key_place(int d) {
  return (d & ~31) + ((d & 15) >> 2) * 8 + ((d >> 4) & 1) * 4 + (d & 3);
}

// E of every piece.  A block of four waves per (piece, head, 64 columns): keys and weighted values lie
// in LDS with their tokens side by side; D[key][column] = K^T V', a wave takes 16 columns.
template <bool VEC>
__global__ __launch_bounds__(256) void state_piece_add_kernel(const ChunkArgs a) {
  extern __shared__ __attribute__((aligned(16))) unsigned char sc_lds[];
  const StateStep& p = a.s;
  const int piece = blockIdx.x, head = blockIdx.y, c0 = blockIdx.z * 64;
  const int t0 = a.piece_cu[piece], count = a.piece_cu[piece + 1] - t0;
  if (count <= 0) return;
  const int columns = p.value_dim + (p.ones ? 1 : 0);
  const int key_rows = (p.key_dim + 15) / 16 * 16;
  float* s_log = reinterpret_cast<float*>(sc_lds);
  float* s_take = s_log + SC_TOKENS;
  bf16_t* s_k = reinterpret_cast<bf16_t*>(s_take + SC_TOKENS);      // [key_rows][SC_ROW]
  bf16_t* s_hi = s_k + key_rows * SC_ROW;                           // [64][SC_ROW]
  bf16_t* s_lo = s_hi + 64 * SC_ROW;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  piece_decays(p, head, t0, count, s_log, s_take);
  __syncthreads();
  // what lies behind the last token is zero
  const float last_log = s_log[SC_TOKENS - 1];
  stage_transposed<VEC>(p.v + (int64_t)t0 * p.v_ld + head * p.value_dim, p.v_ld, count, c0, p.value_dim, 64,
                   [&](int d, int tt, float x0, float x1) {
                     const int c = c0 + d;
                     const bool own = c < p.value_dim;
                     const float other = p.ones && c == p.value_dim ? 1.f : 0.f;
                     const float v0 = (own ? x0 : other) * s_take[tt] * expf(last_log - s_log[tt]);
                     const float v1 = (own ? x1 : other) * s_take[tt + 1] * expf(last_log - s_log[tt + 1]);
                     const uint32_t hi = pack2_bf16(tt < count ? v0 : 0.f, tt + 1 < count ? v1 : 0.f);
                     *reinterpret_cast<uint32_t*>(s_hi + d * SC_ROW + tt) = hi;
                     *reinterpret_cast<uint32_t*>(s_lo + d * SC_ROW + tt) =
                         pack2_bf16(tt < count ? v0 - __uint_as_float(hi << 16) : 0.f,
                                    tt + 1 < count ? v1 - __uint_as_float(hi & 0xffff0000u) : 0.f);
                   });
  stage_transposed<VEC>(p.k + (int64_t)t0 * p.k_ld + (head / p.key_share) * p.key_dim, p.k_ld, count, 0, p.key_dim,
                   key_rows, [&](int d, int tt, float x0, float x1) {
                     const bool own = d < p.key_dim;
                     *reinterpret_cast<uint32_t*>(s_k + d * SC_ROW + tt) =
                         pack2_bf16(own && tt < count ? x0 : 0.f, own && tt + 1 < count ? x1 : 0.f);
                   });
  __syncthreads();
  const int r = lane & 15, g = lane >> 4;
  if (c0 + 16 * wave < columns) {
    bf16x8 hi[2], lo[2];
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      hi[ks] = as_operand(*reinterpret_cast<const uint4*>(s_hi + (16 * wave + r) * SC_ROW + 32 * ks + 8 * g));
      lo[ks] = as_operand(*reinterpret_cast<const uint4*>(s_lo + (16 * wave + r) * SC_ROW + 32 * ks + 8 * g));
    }
    const int c = c0 + 16 * wave + r;
    float* record = a.records + (((int64_t)piece * p.heads + head) * columns + (c < columns ? c : 0)) * p.key_dim;
    for (int n0 = 0; n0 < p.key_dim; n0 += 16) {
      f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        const bf16x8 kf = as_operand(*reinterpret_cast<const uint4*>(s_k + (n0 + r) * SC_ROW + 32 * ks + 8 * g));
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, hi[ks], acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, lo[ks], acc, 0, 0, 0);
      }
      // element i: key 4 g + i, the wave's column r
      const int d = n0 + 4 * g;
      if (c < columns && d < p.key_dim) {
        if (VEC) {
          *reinterpret_cast<float4*>(record + d) = make_float4(acc[0], acc[1], acc[2], acc[3]);
        } else {
#pragma unroll
          for (int i = 0; i < 4; ++i)
            if (d + i < p.key_dim) record[d + i] = acc[i];
        }
      }
    }
  }
  if (blockIdx.z == 0 && threadIdx.x == 0) a.totals[(int64_t)piece * p.heads + head] = s_log[SC_TOKENS - 1];
}

// A thread per four numbers of an item's state (one, where the sizes are odd): the slot's, then piece after
// piece its start goes where the piece's addition was; the last state goes to the slot.  Also keeps the
// convolution's inputs.
template <int VEC>
__global__ __launch_bounds__(256) void state_piece_join_kernel(const ChunkArgs a) {
  const StateStep& p = a.s;
  const int item = blockIdx.x, head = blockIdx.y;
  const int columns = p.value_dim + (p.ones ? 1 : 0);
  const int per_head = columns * p.key_dim;
  const int first = a.item_first[item], last = a.item_first[item + 1];
  if (first == last) return;
  float* slot = p.state + p.slots[item] * p.slot_stride;
  const int e = (blockIdx.z * 256 + threadIdx.x) * VEC;
  if (e < per_head) {
    float* mine = slot + (int64_t)head * per_head + e;
    float* record = a.records + ((int64_t)first * p.heads + head) * per_head + e;
    const int64_t step = (int64_t)p.heads * per_head;
    float s[VEC], left[VEC];
#pragma unroll
    for (int i = 0; i < VEC; ++i) s[i] = mine[i];
#pragma unroll
    for (int i = 0; i < VEC; ++i) left[i] = record[i];
    for (int k = first; k < last; ++k) {
      const float keep = expf(a.totals[(int64_t)k * p.heads + head]);
      float next[VEC];
      // the next piece's addition is on its way meanwhile
      const float* ahead = record + (k + 1 < last ? step : 0);
#pragma unroll
      for (int i = 0; i < VEC; ++i) next[i] = ahead[i];
#pragma unroll
      for (int i = 0; i < VEC; ++i) {
        record[i] = s[i];
        s[i] = fmaf(keep, s[i], left[i]);
        left[i] = next[i];
      }
      record += step;
    }
#pragma unroll
    for (int i = 0; i < VEC; ++i) mine[i] = s[i];
  }
  state_keep_inputs(p, slot, p.cu_tokens[item], p.cu_tokens[item + 1],
                    (blockIdx.y * gridDim.z + blockIdx.z) * 256 + threadIdx.x, gridDim.y * gridDim.z * 256);
}

// The outputs.  A block of four waves per (piece, head, 16 NT columns); a wave takes 16 tokens as the columns
// of its products: O^T[column][token] = e^(L_t) (S0^T Q^T) + V^T P^T, P^T[s][t] = K Q^T with the decays between
// the tokens, their weights and the mask.  Operands: queries and states from memory as they lie (twice 4
// consecutive key dimensions a lane), keys from LDS in the same order, values from LDS with the tokens side
// by side.
// A lane holds P^T of four consecutive tokens s per tile of 16; two such tiles fill the eight places of
// its operand of the next product, and the values are read in the same order.
template <int NT, int KS, bool VEC>
__global__ __launch_bounds__(256) void state_piece_out_kernel(const ChunkArgs a) {
  extern __shared__ __attribute__((aligned(16))) unsigned char sc_lds[];
  const StateStep& p = a.s;
  const int piece = blockIdx.x, head = blockIdx.y, c0 = blockIdx.z * 16 * NT;
  const int t0 = a.piece_cu[piece], count = a.piece_cu[piece + 1] - t0;
  if (count <= 0) return;
  const int columns = p.value_dim + (p.ones ? 1 : 0);
  constexpr int key_row = 32 * KS + 8;
  float* s_log = reinterpret_cast<float*>(sc_lds);
  float* s_take = s_log + SC_TOKENS;
  bf16_t* s_k = reinterpret_cast<bf16_t*>(s_take + SC_TOKENS);      // [SC_TOKENS][key_row]
  bf16_t* s_v = s_k + SC_TOKENS * key_row;                          // [16 NT][SC_ROW]
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r = lane & 15, g = lane >> 4;
  const int key_head = head / p.key_share;
  const int tq = 16 * wave + r;                  // the lane's token
  piece_decays(p, head, t0, count, s_log, s_take);
  // the lane's query: 8 dimensions of every 32
  bf16x8 qf[KS];
  {
    const float* q_row = p.q + (int64_t)(t0 + (tq < count ? tq : count - 1)) * p.q_ld + key_head * p.key_dim;
    float x[KS][8];
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      piece_four<VEC>(q_row, 32 * ks + 4 * g, p.key_dim, &x[ks][0]);
      piece_four<VEC>(q_row, 32 * ks + 16 + 4 * g, p.key_dim, &x[ks][4]);
    }
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      uint32_t qw[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = 32 * ks + 16 * (i >> 1) + 4 * g + 2 * (i & 1);
        qw[i] = pack2_bf16(d < p.key_dim ? x[ks][2 * i] : 0.f, d + 1 < p.key_dim ? x[ks][2 * i + 1] : 0.f);
      }
      qf[ks] = as_operand(make_uint4(qw[0], qw[1], qw[2], qw[3]));
    }
  }
  // the keys of 16 tokens of every wave, 64 dimensions of a token side by side
  for (int d = lane; d < 32 * KS; d += 64) {
    float x[16];
    const float* k_col = p.k + key_head * p.key_dim + (d < p.key_dim ? d : 0);
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int tt = 16 * wave + i < count ? 16 * wave + i : count - 1;
      x[i] = k_col[(int64_t)(t0 + tt) * p.k_ld];
    }
#pragma unroll
    for (int i = 0; i < 16; ++i)
      s_k[(16 * wave + i) * key_row + key_place(d)] = float_to_bf16(16 * wave + i < count && d < p.key_dim ? x[i] : 0.f);
  }
  stage_transposed<VEC>(p.v + (int64_t)t0 * p.v_ld + head * p.value_dim, p.v_ld, count, c0, p.value_dim, 16 * NT,
                   [&](int d, int tt, float x0, float x1) {
                     const int c = c0 + d;
                     const bool own = c < p.value_dim;
                     const float other = p.ones && c == p.value_dim ? 1.f : 0.f;
                     *reinterpret_cast<uint32_t*>(s_v + d * SC_ROW + tt) =
                         pack2_bf16(tt < count ? (own ? x0 : other) : 0.f, tt + 1 < count ? (own ? x1 : other) : 0.f);
                   });
  __syncthreads();
  if (16 * wave >= count) return;                // (a whole wave, behind the last barrier)
  const float* start = a.records + ((int64_t)piece * p.heads + head) * columns * p.key_dim;
  f32x4 acc[NT], pt[4];
#pragma unroll
  for (int n = 0; n < NT; ++n) acc[n] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int k = 0; k < 4; ++k) pt[k] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) {
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      if (k <= wave) {
        const bf16x8 kf = as_operand(*reinterpret_cast<const uint4*>(s_k + (16 * k + r) * key_row + 32 * ks + 8 * g));
        pt[k] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[ks], pt[k], 0, 0, 0);
      }
    }
    float s[NT][8];
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      const int c = c0 + 16 * n + r < columns ? c0 + 16 * n + r : columns - 1;
      piece_four<VEC>(start + (int64_t)c * p.key_dim, 32 * ks + 4 * g, p.key_dim, &s[n][0]);
      piece_four<VEC>(start + (int64_t)c * p.key_dim, 32 * ks + 16 + 4 * g, p.key_dim, &s[n][4]);
    }
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      uint32_t hw[4], lw[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        // (a query's places behind its own size are zero: what stands against them does not matter, but
        // must be finite)
        hw[i] = pack2_bf16(s[n][2 * i], s[n][2 * i + 1]);
        lw[i] = pack2_bf16(s[n][2 * i] - __uint_as_float(hw[i] << 16), s[n][2 * i + 1] - __uint_as_float(hw[i] & 0xffff0000u));
      }
      const uint4 hv = make_uint4(hw[0], hw[1], hw[2], hw[3]), lv = make_uint4(lw[0], lw[1], lw[2], lw[3]);
      acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_operand(hv), qf[ks], acc[n], 0, 0, 0);
      acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_operand(lv), qf[ks], acc[n], 0, 0, 0);
    }
  }
  // element i of a lane: row 4 g + i (a column of the values, or token s of a tile), token tq
  const float log_q = s_log[tq];
  const float kept = expf(log_q);
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[n][i] *= kept;
#pragma unroll
  for (int pair = 0; pair < 2; ++pair) {
    if (2 * pair > wave) break;                  // (the same in every lane of the wave)
    uint32_t hw[4], lw[4];
#pragma unroll
    for (int half = 0; half < 2; ++half) {
      float w[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int ts = 16 * (2 * pair + half) + 4 * g + i;
        w[i] = ts <= tq ? pt[2 * pair + half][i] * s_take[ts] * expf(log_q - s_log[ts]) : 0.f;
      }
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const uint32_t hi = pack2_bf16(w[2 * i], w[2 * i + 1]);
        hw[2 * half + i] = hi;
        lw[2 * half + i] = pack2_bf16(w[2 * i] - __uint_as_float(hi << 16), w[2 * i + 1] - __uint_as_float(hi & 0xffff0000u));
      }
    }
    const uint4 hv = make_uint4(hw[0], hw[1], hw[2], hw[3]), lv = make_uint4(lw[0], lw[1], lw[2], lw[3]);
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      const bf16_t* from = s_v + (16 * n + r) * SC_ROW + 32 * pair + 4 * g;
      const uint2 low = *reinterpret_cast<const uint2*>(from), high = *reinterpret_cast<const uint2*>(from + 16);
      const uint4 vv = make_uint4(low.x, low.y, high.x, high.y);
      acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_operand(vv), as_operand(hv), acc[n], 0, 0, 0);
      acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_operand(vv), as_operand(lv), acc[n], 0, 0, 0);
    }
  }
  if (tq >= count) return;
  float* out = p.out + ((int64_t)(t0 + tq) * p.heads + head) * columns;
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    const int c = c0 + 16 * n + 4 * g;
    if (VEC && columns % 4 == 0) {
      if (c < columns)
        *reinterpret_cast<float4*>(out + c) = make_float4(acc[n][0] * p.q_scale, acc[n][1] * p.q_scale,
                                                          acc[n][2] * p.q_scale, acc[n][3] * p.q_scale);
      continue;
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (c + i < columns) out[c + i] = acc[n][i] * p.q_scale;
  }
}

extern "C" int ps_state_chunk_tokens() { return SC_TOKENS; }

extern "C" int ps_state_chunks(const float* q, int64_t q_ld, const float* k, int64_t k_ld, const float* v,
                               int64_t v_ld, const float* decay, const float* take, float* state,
                               int64_t slot_stride, float* out, const int* cu_tokens, const int* slots,
                               int items, int heads, int key_share, int key_dim, int value_dim, int ones,
                               float q_scale, const float* raw, int64_t raw_ld, int channels, int taps,
                               int64_t history, const int* piece_cu, const int* item_first, int pieces,
                               float* records, int64_t records_floats, float* totals, void* stream) {
  PS_REQUIRE(items >= 0 && heads > 0 && key_share > 0 && heads % key_share == 0 && key_dim > 0 && value_dim > 0 &&
                 pieces >= 0,
             "ps_state_chunks: bad sizes");
  PS_REQUIRE(key_dim <= 256 && heads <= 65535, "ps_state_chunks: key head size %d above 256", key_dim);
  PS_REQUIRE(channels == 0 || (raw != nullptr && taps >= 1), "ps_state_chunks: the convolution's inputs are missing");
  const int columns = value_dim + (ones ? 1 : 0);
  const int64_t need = (int64_t)pieces * heads * columns * key_dim;
  PS_REQUIRE(records != nullptr && totals != nullptr && records_floats >= need,
             "ps_state_chunks: the records need %lld floats", (long long)need);
  if (items == 0 || pieces == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const int aligned = (uintptr_t)records % 16 == 0;
  // rows of queries, keys and values that allow loads of 16 bytes
  const int vectors = aligned && key_dim % 4 == 0 && value_dim % 4 == 0 && q_ld % 4 == 0 && k_ld % 4 == 0 && v_ld % 4 == 0 &&
                      (uintptr_t)q % 16 == 0 && (uintptr_t)k % 16 == 0 && (uintptr_t)v % 16 == 0 && (uintptr_t)out % 16 == 0;
  const ChunkArgs a = {{q, q_ld, k, k_ld, v, v_ld, decay, take, state, slot_stride, out, cu_tokens, slots, heads,
                        key_share, key_dim, value_dim, ones, q_scale, aligned, vectors, raw, raw_ld, channels, taps, history},
                       piece_cu, item_first, records, totals};
  const int key_rows = (key_dim + 15) / 16 * 16;
  const size_t add_lds = 2 * SC_TOKENS * sizeof(float) + (size_t)(key_rows + 128) * SC_ROW * sizeof(bf16_t);
  if (vectors)
    hipLaunchKernelGGL(state_piece_add_kernel<true>, dim3(pieces, heads, (columns + 63) / 64), dim3(256), add_lds, s, a);
  else
    hipLaunchKernelGGL(state_piece_add_kernel<false>, dim3(pieces, heads, (columns + 63) / 64), dim3(256), add_lds, s, a);
  PS_CHECK_LAUNCH("ps_state_chunks(add)");
  const int per_head = columns * key_dim;
  const bool four = per_head % 4 == 0 && aligned && slot_stride % 4 == 0 && (uintptr_t)state % 16 == 0;
  if (four)
    hipLaunchKernelGGL(state_piece_join_kernel<4>, dim3(items, heads, (per_head / 4 + 255) / 256), dim3(256), 0, s, a);
  else
    hipLaunchKernelGGL(state_piece_join_kernel<1>, dim3(items, heads, (per_head + 255) / 256), dim3(256), 0, s, a);
  PS_CHECK_LAUNCH("ps_state_chunks(join)");
#define PS_LAUNCH_SPO_V(NT, KS, VEC)                                                                       \
  hipLaunchKernelGGL((state_piece_out_kernel<NT, KS, VEC>), dim3(pieces, heads, (columns + 16 * NT - 1) / (16 * NT)), dim3(256), \
                     2 * SC_TOKENS * sizeof(float) + ((size_t)SC_TOKENS * (32 * KS + 8) + 16 * NT * SC_ROW) * sizeof(bf16_t), s, a)
#define PS_LAUNCH_SPO_K(NT, KS)                     \
  do {                                              \
    if (vectors) PS_LAUNCH_SPO_V(NT, KS, true);     \
    else PS_LAUNCH_SPO_V(NT, KS, false);            \
  } while (0)
#define PS_LAUNCH_SPO(NT)                           \
  do {                                              \
    if (key_dim <= 64) PS_LAUNCH_SPO_K(NT, 2);      \
    else if (key_dim <= 128) PS_LAUNCH_SPO_K(NT, 4); \
    else PS_LAUNCH_SPO_K(NT, 8);                    \
  } while (0)
  if (columns <= 32) PS_LAUNCH_SPO(2);
  else if (columns <= 64) PS_LAUNCH_SPO(4);
  else if (columns <= 80) PS_LAUNCH_SPO(5);
  else PS_LAUNCH_SPO(4);
#undef PS_LAUNCH_SPO
#undef PS_LAUNCH_SPO_K
#undef PS_LAUNCH_SPO_V
  PS_CHECK_LAUNCH("ps_state_chunks(out)");
  return 0;
}
