// Recurrent mixers whose state is a matrix per head, S: [key_dim, value_dim] in float per request,
// read by a query as o = S^T q.  Two rules move it from token to token:
//
//   decayed   S_t = e^(l_t) S_(t-1) + w_t k_t v_t^T            one decay and one weight per head
//   delta     S' = diag(g_t) S_(t-1),  S_t = S' + w_t k_t (v_t - S'^T k_t)^T      a decay per key channel
//
// (state spaces with a decay per head, matrix memories with exponential gates, the gated delta rule).
// A slot's state is one run of floats: the heads' matrices, stored value column by value column
// ([head][column][key row]), and behind them whatever else the mixer keeps: the last taps - 1 raw
// inputs of its short convolution ([taps - 1][channels], oldest first), a running maximum per head.
//
// Launches of a step: what the recurrence is fed with (ps_state_prepare: convolutions, unit norms,
// decays, weights; or ps_memory_gates), the recurrence, and the norm and gate of its output
// (ps_state_output).  All of it is 32-bit; only the last launch writes the engine's type.
#include <math.h>

#include "common.h"
#include "matrix_state.h"
#include "pagedserve_hip.h"

__device__ inline float ms_silu(float v) { return v / (1.0f + expf(-v)); }
__device__ inline float ms_sigmoid(float v) { return 1.0f / (1.0f + expf(-v)); }
// softplus(v) = max(v, 0) + log1p(exp(-|v|))
__device__ inline float ms_softplus(float v) { return fmaxf(v, 0.f) + log1pf(expf(-fabsf(v))); }

// ---- short convolutions and what goes with them ------------------------------------------------
// A wave per unit of a token.  Units of the convolution: the first `unit_heads` runs of `head`
// channels each, whose activated values are made unit vectors (the first `scale_heads` of them are
// also multiplied by q_scale), then runs of 256 of the other channels.  Then units of 256 decays.
#define MS_UNIT 256
struct PrepareArgs {
  const float* proj;
  int64_t ld;
  int col, channels, taps;
  const float* w;          // [channels, taps], the last column is the current token's
  const float* bias;       // [channels] or null
  const float* state;
  int64_t slot_stride;
  int64_t history;         // where a slot's kept inputs begin
  float* out;              // [tokens, channels]
  int unit_heads, head, scale_heads;
  float q_scale;
  int rule;                // PS_STATE_DECAYED or PS_STATE_DELTA
  int heads, per_head;     // decays: heads (decayed) or heads * per_head (delta) per token
  const float* z;          // delta: rows of raw decays
  int64_t z_ld;
  const float* z_bias;     // per decay
  const float* a_log;      // per head
  int take_col;            // columns of proj that give the weights (delta) or steps (decayed)
  float* decay;            // [tokens, heads] logarithms (decayed), [tokens, heads * per_head] factors (delta)
  float* take;             // [tokens, heads]
  const int* tok_item;
  const int* cu_tokens;
  const int* slots;
  int conv_units, decay_units;
};

__global__ __launch_bounds__(256) void state_prepare_kernel(const PrepareArgs p) {
  const int t = blockIdx.x;
  const int lane = threadIdx.x & 63;
  const int unit = blockIdx.y * 4 + (threadIdx.x >> 6);
  if (unit >= p.conv_units + p.decay_units) return;
  const float* row = p.proj + (int64_t)t * p.ld;
  if (unit >= p.conv_units) {
    const int first = (unit - p.conv_units) * MS_UNIT;
    const int count = p.rule == PS_STATE_DELTA ? p.heads * p.per_head : p.heads;
#pragma unroll
    for (int j = 0; j < MS_UNIT / 64; ++j) {
      const int c = first + j * 64 + lane;
      if (c < p.heads) {
        const float raw = row[p.take_col + c];
        if (p.rule == PS_STATE_DELTA) {
          p.take[(int64_t)t * p.heads + c] = ms_sigmoid(raw);
        } else {
          const float dt = ms_softplus(raw + p.z_bias[c]);
          p.take[(int64_t)t * p.heads + c] = dt;
          p.decay[(int64_t)t * p.heads + c] = -expf(p.a_log[c]) * dt;
        }
      }
      if (p.rule == PS_STATE_DELTA && c < count) {
        const float step = ms_softplus(p.z[(int64_t)t * p.z_ld + c] + p.z_bias[c]);
        p.decay[(int64_t)t * count + c] = expf(-expf(p.a_log[c / p.per_head]) * step);
      }
    }
    return;
  }
  const bool normed = unit < p.unit_heads;
  const int c0 = normed ? unit * p.head : p.unit_heads * p.head + (unit - p.unit_heads) * MS_UNIT;
  const int most = normed ? p.head : MS_UNIT;
  const int count = p.channels - c0 < most ? p.channels - c0 : most;
  const int item = p.tok_item[t];
  const int first = p.cu_tokens[item];
  const float* kept = p.state + p.slots[item] * p.slot_stride + p.history;
  float value[4], squares = 0.f;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int d = j * 64 + lane;
    value[j] = 0.f;
    if (d < count) {
      const int c = c0 + d;
      float sum = p.bias ? p.bias[c] : 0.f;
      for (int tap = 0; tap < p.taps; ++tap) {
        const int back = p.taps - 1 - tap;          // the input `back` tokens before this one
        const int local = (t - first) - back;       // its place among the item's tokens of this step
        const float u = local >= 0 ? row[p.col + c - (int64_t)back * p.ld]
                                   : kept[(int64_t)(p.taps - 1 + local) * p.channels + c];
        sum = fmaf(p.w[(int64_t)c * p.taps + tap], u, sum);
      }
      value[j] = ms_silu(sum);
    }
    squares = fmaf(value[j], value[j], squares);
  }
  float factor = 1.f;
  if (normed) {
    factor = 1.0f / sqrtf(wave_sum(squares) + 1e-6f);
    if (unit < p.scale_heads) factor *= p.q_scale;
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int d = j * 64 + lane;
    if (d < count) p.out[(int64_t)t * p.channels + c0 + d] = value[j] * factor;
  }
}

extern "C" int ps_state_prepare(const float* proj, int64_t ld, int col, int channels, int taps,
                                const float* w, const float* bias, const float* state,
                                int64_t slot_stride, int64_t history, float* out, int unit_heads,
                                int head, int scale_heads, float q_scale, int rule, int heads,
                                int per_head, const float* z, int64_t z_ld, const float* z_bias,
                                const float* a_log, int take_col, float* decay, float* take,
                                const int* tok_item, const int* cu_tokens, const int* slots, int tokens,
                                void* stream) {
  PS_REQUIRE(tokens >= 0 && channels > 0 && taps >= 1 && taps <= 64 && heads > 0 && per_head > 0,
             "ps_state_prepare: bad sizes");
  PS_REQUIRE(unit_heads >= 0 && (int64_t)unit_heads * head <= channels && scale_heads <= unit_heads &&
                 (unit_heads == 0 || (head > 0 && head <= MS_UNIT)),
             "ps_state_prepare: %d heads of %d do not fit %d channels (heads of up to %d)", unit_heads, head,
             channels, MS_UNIT);
  PS_REQUIRE(rule == PS_STATE_DECAYED || (rule == PS_STATE_DELTA && z != nullptr),
             "ps_state_prepare: rule %d", rule);
  if (tokens == 0) return 0;
  PrepareArgs p = {proj, ld, col, channels, taps, w, bias, state, slot_stride, history, out, unit_heads,
                   head, scale_heads, q_scale, rule, heads, per_head, z, z_ld, z_bias, a_log, take_col,
                   decay, take, tok_item, cu_tokens, slots, 0, 0};
  p.conv_units = unit_heads + (channels - unit_heads * head + MS_UNIT - 1) / MS_UNIT;
  const int decays = rule == PS_STATE_DELTA ? heads * per_head : heads;
  p.decay_units = (decays + MS_UNIT - 1) / MS_UNIT;
  const int units = p.conv_units + p.decay_units;
  PS_REQUIRE((units + 3) / 4 <= 65535, "ps_state_prepare: too many channels");
  hipLaunchKernelGGL(state_prepare_kernel, dim3(tokens, (units + 3) / 4), dim3(256), 0, (hipStream_t)stream, p);
  PS_CHECK_LAUNCH("ps_state_prepare");
  return 0;
}

// ---- gates of a matrix memory ---------------------------------------------------------------------
// Per head, with raw gates a and b: i = cap tanh(a / cap), f = log sigmoid(cap tanh(b / cap)); the
// running maximum m_t = max(f + m_(t-1), i) starts at the slot's; what the recurrence needs is
// l_t = f + m_(t-1) - m_t, w_t = e^(i - m_t) and, for the output, e^(-m_t).  A wave per (item, head):
// 64 tokens at a time, the maps m -> max(f + m, i) composed over the lanes.
__global__ __launch_bounds__(64) void memory_gates_kernel(
    const float* __restrict__ proj, int64_t ld, int i_col, int f_col, const float* __restrict__ i_bias,
    const float* __restrict__ f_bias, float cap, float* __restrict__ state, int64_t slot_stride,
    int64_t maxima, float* __restrict__ log_decay, float* __restrict__ take, float* __restrict__ floor_out,
    const int* __restrict__ cu_tokens, const int* __restrict__ slots, int heads) {
  const int item = blockIdx.x, head = blockIdx.y, lane = threadIdx.x;
  const int t0 = cu_tokens[item], t1 = cu_tokens[item + 1];
  if (t0 >= t1) return;
  float* kept = state + slots[item] * slot_stride + maxima + head;
  float m = *kept;
  const float ib = i_bias[head], fb = f_bias[head];
  auto place = [&](const int base) { return (int64_t)(base + lane < t1 ? base + lane : t1 - 1); };
  float raw_i = proj[place(t0) * ld + i_col + head], raw_f = proj[place(t0) * ld + f_col + head];
  for (int base = t0; base < t1; base += 64) {
    const float i = cap * tanhf((raw_i + ib) / cap);
    const float capped = cap * tanhf((raw_f + fb) / cap);
    const float f = fminf(capped, 0.f) - log1pf(expf(-fabsf(capped)));
    if (base + 64 < t1) {
      // the next 64 are on their way during the work below
      raw_i = proj[place(base + 64) * ld + i_col + head];
      raw_f = proj[place(base + 64) * ld + f_col + head];
    }
    // lane n: the composition of the maps of lanes 0 .. n is m -> max(add + m, least)
    float add = f, least = i;
#pragma unroll
    for (int step = 1; step < 64; step <<= 1) {
      const float add_before = __shfl_up(add, step, 64);
      const float least_before = __shfl_up(least, step, 64);
      if (lane >= step) {
        least = fmaxf(add + least_before, least);
        add += add_before;
      }
    }
    const float after = fmaxf(add + m, least);
    float before = __shfl_up(after, 1, 64);
    if (lane == 0) before = m;
    const int count = t1 - base < 64 ? t1 - base : 64;
    if (lane < count) {
      const int64_t at = (int64_t)(base + lane) * heads + head;
      log_decay[at] = f + before - after;
      take[at] = expf(i - after);
      floor_out[at] = expf(-after);
    }
    m = __shfl(after, count - 1, 64);
  }
  if (lane == 0) *kept = m;
}

extern "C" int ps_memory_gates(const float* proj, int64_t ld, int i_col, int f_col, const float* i_bias,
                               const float* f_bias, float cap, float* state, int64_t slot_stride,
                               int64_t maxima, float* log_decay, float* take, float* floor_out,
                               const int* cu_tokens, const int* slots, int items, int heads,
                               void* stream) {
  PS_REQUIRE(items >= 0 && heads > 0 && heads <= 65535 && cap > 0.f, "ps_memory_gates: bad sizes");
  if (items == 0) return 0;
  hipLaunchKernelGGL(memory_gates_kernel, dim3(items, heads), dim3(64), 0, (hipStream_t)stream, proj, ld,
                     i_col, f_col, i_bias, f_bias, cap, state, slot_stride, maxima, log_decay, take,
                     floor_out, cu_tokens, slots, heads);
  PS_CHECK_LAUNCH("ps_memory_gates");
  return 0;
}

// ---- the recurrence, token after token --------------------------------------------------------------
// A block of four waves owns 4 COLS columns of one head's state for one item.  Within a wave, lane =
// column * GROUPS + row group; a lane keeps RPL neighbouring key rows of its column in registers, and
// the sums over the row groups run over neighbouring lanes.  Keys, queries, decays and values of
// MS_CHUNK tokens wait in LDS for all four waves; the next chunk's loads travel while this one is
// worked on.

template <int RPL, int GROUPS, int CHUNK, bool DELTA>
__global__ __launch_bounds__(256) void state_walk_kernel(const StateStep p) {
  constexpr int COLS = 64 / GROUPS;                // columns of a wave
  constexpr int BLOCK_COLS = 4 * COLS;
  constexpr int ROWS = GROUPS * RPL;               // key rows with padding up to the lanes' share
  constexpr int PAD = RPL < 4 ? 4 : RPL + 4;       // row groups start in different banks
  constexpr int PER = (CHUNK * ROWS + 255) / 256;  // values of a chunk per thread and array
  constexpr int PER_V = (CHUNK * BLOCK_COLS + 255) / 256;
  __shared__ __attribute__((aligned(16))) float s_q[CHUNK][GROUPS * PAD];
  __shared__ __attribute__((aligned(16))) float s_k[CHUNK][GROUPS * PAD];
  __shared__ __attribute__((aligned(16))) float s_a[DELTA ? CHUNK : 1][GROUPS * PAD];
  __shared__ float s_v[CHUNK][BLOCK_COLS];
  __shared__ float s_o[CHUNK][BLOCK_COLS];
  __shared__ float s_d[CHUNK], s_w[CHUNK];
  const int item = blockIdx.x, head = blockIdx.y;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int group = lane % GROUPS;
  const int mine = wave * COLS + lane / GROUPS;    // the lane's column within the block
  const int col0 = blockIdx.z * BLOCK_COLS;
  const int col = col0 + mine;
  const int columns = p.value_dim + (p.ones ? 1 : 0);
  const bool has_col = col < columns;
  const int t0 = p.cu_tokens[item], t1 = p.cu_tokens[item + 1];
  if (t0 >= t1) return;
  float* slot = p.state + p.slots[item] * p.slot_stride;
  float* s_ptr = slot + ((int64_t)head * columns + (has_col ? col : 0)) * p.key_dim + group * RPL;
  const int key_head = head / p.key_share;
  const float* k_base = p.k + key_head * p.key_dim;
  const float* q_base = p.q + key_head * p.key_dim;
  const float* v_base = p.v + head * p.value_dim;
  const float* a_base = DELTA ? p.decay + (int64_t)head * p.key_dim : nullptr;
  const int64_t a_ld = (int64_t)p.heads * p.key_dim;
  float S[RPL];
  const int rows_mine = p.key_dim - group * RPL;   // key rows from the lane's first on
  const bool whole = RPL % 4 == 0 && p.key_dim % 4 == 0 && p.aligned;
  if (whole) {
#pragma unroll
    for (int i = 0; i < RPL; i += 4) {
      float4 four = make_float4(0.f, 0.f, 0.f, 0.f);
      if (i < rows_mine && has_col) four = *reinterpret_cast<const float4*>(s_ptr + i);
      S[i] = four.x;
      if (RPL >= 4) {
        S[(i + 1) % RPL] = four.y;
        S[(i + 2) % RPL] = four.z;
        S[(i + 3) % RPL] = four.w;
      }
    }
  } else {
#pragma unroll
    for (int i = 0; i < RPL; ++i) S[i] = (i < rows_mine && has_col) ? s_ptr[i] : 0.f;
  }
  float rq[PER], rk[PER], ra[DELTA ? PER : 1], rv[PER_V], rd = 0.f, rw = 0.f;
  // every load is unconditional from a clamped address; what lies outside is masked when stored
  auto fetch = [&](const int base) {
    const int count = (t1 - base) < CHUNK ? (t1 - base) : CHUNK;
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int idx = tid + j * 256;
      const int tt = idx / ROWS;
      const int r = idx - tt * ROWS;
      const int64_t t = base + (tt < count ? tt : 0);
      const int c = r < p.key_dim ? r : 0;
      rq[j] = q_base[t * p.q_ld + c];
      rk[j] = k_base[t * p.k_ld + c];
      if (DELTA) ra[j] = a_base[t * a_ld + c];
    }
#pragma unroll
    for (int j = 0; j < PER_V; ++j) {
      const int idx = tid + j * 256;
      const int tt = idx / BLOCK_COLS;
      const int c = col0 + (idx - tt * BLOCK_COLS);
      const int64_t t = base + (tt < count ? tt : 0);
      rv[j] = v_base[t * p.v_ld + (c < p.value_dim ? c : 0)];
    }
    if (tid < CHUNK) {
      const int64_t at = (int64_t)(base + (tid < count ? tid : 0)) * p.heads + head;
      rw = p.take[at];
      if (!DELTA) rd = p.decay[at];
    }
  };
  auto stash = [&](const int base) {
    const int count = (t1 - base) < CHUNK ? (t1 - base) : CHUNK;
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int idx = tid + j * 256;
      const int tt = idx / ROWS;
      const int r = idx - tt * ROWS;
      const bool valid = tt < count && r < p.key_dim;
      const int at = (r / RPL) * PAD + (r % RPL);
      if (CHUNK * ROWS % 256 == 0 || tt < CHUNK) {
        s_q[tt][at] = valid ? rq[j] * p.q_scale : 0.f;
        s_k[tt][at] = valid ? rk[j] : 0.f;
        if (DELTA) s_a[tt][at] = valid ? ra[j] : 0.f;
      }
    }
#pragma unroll
    for (int j = 0; j < PER_V; ++j) {
      const int idx = tid + j * 256;
      const int tt = idx / BLOCK_COLS;
      if (CHUNK * BLOCK_COLS % 256 == 0 || tt < CHUNK) {
        const int c = col0 + (idx - tt * BLOCK_COLS);
        // (the column behind the values sums the keys alone: its value is one)
        const float v = c < p.value_dim ? rv[j] : (p.ones && c == p.value_dim ? 1.f : 0.f);
        s_v[tt][idx - tt * BLOCK_COLS] = tt < count ? v : 0.f;
      }
    }
    if (tid < CHUNK) {
      s_w[tid] = rw;
      s_d[tid] = DELTA ? 0.f : expf(rd);
    }
  };
  fetch(t0);
  for (int base = t0; base < t1; base += CHUNK) {
    const int count = (t1 - base) < CHUNK ? (t1 - base) : CHUNK;
    __syncthreads();      // the chunk before has been read
    stash(base);
    __syncthreads();
    if (base + CHUNK < t1) fetch(base + CHUNK);   // in flight during the work below
    auto token = [&](const int tt) {
      const float* kr = &s_k[tt][group * PAD];
      const float* qr = &s_q[tt][group * PAD];
      float v = s_v[tt][mine];
      const float w = s_w[tt];
      if (DELTA) {
        const float* ar = &s_a[tt][group * PAD];
        float dot0 = 0.f, dot1 = 0.f;
#pragma unroll
        for (int i = 0; i < RPL; ++i) {
          S[i] *= ar[i];
          if (i & 1) dot1 = fmaf(S[i], kr[i], dot1);
          else dot0 = fmaf(S[i], kr[i], dot0);
        }
        v = w * (v - lanes_sum<GROUPS>(dot0 + dot1));
      } else {
        const float d = s_d[tt];
        v *= w;
#pragma unroll
        for (int i = 0; i < RPL; ++i) S[i] *= d;
      }
      float o0 = 0.f, o1 = 0.f;
#pragma unroll
      for (int i = 0; i < RPL; ++i) {
        S[i] = fmaf(kr[i], v, S[i]);
        if (i & 1) o1 = fmaf(S[i], qr[i], o1);
        else o0 = fmaf(S[i], qr[i], o0);
      }
      const float o = lanes_sum<GROUPS>(o0 + o1);
      if (group == 0) s_o[tt][mine] = o;
    };
    if (count == CHUNK) {
      // a whole chunk: unrolled, so that the reads of the next tokens run ahead of the chain
#pragma unroll
      for (int tt = 0; tt < CHUNK; ++tt) token(tt);
    } else {
      for (int tt = 0; tt < count; ++tt) token(tt);
    }
    __syncthreads();
    for (int idx = tid; idx < count * BLOCK_COLS; idx += 256) {
      const int tt = idx / BLOCK_COLS;
      const int c = idx - tt * BLOCK_COLS;
      if (col0 + c < columns)
        p.out[((int64_t)(base + tt) * p.heads + head) * columns + col0 + c] = s_o[tt][c];
    }
  }
  if (has_col) {
    if (whole) {
#pragma unroll
      for (int i = 0; i < RPL; i += 4)
        if (i < rows_mine)
          *reinterpret_cast<float4*>(s_ptr + i) = make_float4(S[i], S[(i + 1) % RPL], S[(i + 2) % RPL], S[(i + 3) % RPL]);
    } else {
#pragma unroll
      for (int i = 0; i < RPL; ++i)
        if (i < rows_mine) s_ptr[i] = S[i];
    }
  }
  // the convolution's inputs for the next step: the item's blocks share the channels
  state_keep_inputs(p, slot, t0, t1, (blockIdx.y * gridDim.z + blockIdx.z) * 256 + tid, gridDim.y * gridDim.z * 256);
}

extern "C" int ps_state_scan(const float* q, int64_t q_ld, const float* k, int64_t k_ld, const float* v,
                             int64_t v_ld, const float* decay, const float* take, float* state,
                             int64_t slot_stride, float* out, const int* cu_tokens, const int* slots,
                             int items, int rule, int heads, int key_share, int key_dim, int value_dim,
                             int ones, float q_scale, int longest, const float* raw, int64_t raw_ld,
                             int channels, int taps, int64_t history, void* stream) {
  PS_REQUIRE(items >= 0 && heads > 0 && key_share > 0 && heads % key_share == 0 && key_dim > 0 && value_dim > 0,
             "ps_state_scan: bad sizes");
  PS_REQUIRE(key_dim <= 256, "ps_state_scan: key head size %d above 256", key_dim);
  PS_REQUIRE(rule == PS_STATE_DECAYED || (rule == PS_STATE_DELTA && !ones), "ps_state_scan: rule %d", rule);
  PS_REQUIRE(channels == 0 || (raw != nullptr && taps >= 1), "ps_state_scan: the convolution's inputs are missing");
  const int columns = value_dim + (ones ? 1 : 0);
  PS_REQUIRE(heads <= 65535 && (columns + 15) / 16 <= 65535, "ps_state_scan: grid too large");
  if (items == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const int aligned = slot_stride % 4 == 0 && (uintptr_t)state % 16 == 0;
  const StateStep p = {q, q_ld, k, k_ld, v, v_ld, decay, take, state, slot_stride, out, cu_tokens, slots,
                       heads, key_share, key_dim, value_dim, ones, q_scale, aligned, raw, raw_ld, channels, taps,
                       history};
  const bool brief = longest == 1;
#define PS_LAUNCH_WALK_D(RPL, GROUPS, CHUNK, DELTA)                                               \
  hipLaunchKernelGGL((state_walk_kernel<RPL, GROUPS, CHUNK, DELTA>),                              \
                     dim3(items, heads, (columns + 256 / GROUPS - 1) / (256 / GROUPS)), dim3(256), 0, s, p)
#define PS_LAUNCH_WALK(RPL, GROUPS, CHUNK)                  \
  do {                                                      \
    if (rule == PS_STATE_DELTA) {                           \
      if (brief) PS_LAUNCH_WALK_D(RPL, GROUPS, 2, true);    \
      else PS_LAUNCH_WALK_D(RPL, GROUPS, CHUNK, true);      \
    } else {                                                \
      if (brief) PS_LAUNCH_WALK_D(RPL, GROUPS, 2, false);   \
      else PS_LAUNCH_WALK_D(RPL, GROUPS, CHUNK, false);     \
    }                                                       \
  } while (0)
  if (key_dim <= 16) PS_LAUNCH_WALK(4, 4, 32);
  else if (key_dim <= 32) PS_LAUNCH_WALK(4, 8, 32);
  else if (key_dim <= 64) PS_LAUNCH_WALK(4, 16, 32);
  else if (key_dim <= 128) PS_LAUNCH_WALK(8, 16, 16);
  else PS_LAUNCH_WALK(16, 16, 8);
#undef PS_LAUNCH_WALK
#undef PS_LAUNCH_WALK_D
  PS_CHECK_LAUNCH("ps_state_scan");
  return 0;
}

// ---- the recurrence's output ---------------------------------------------------------------------
// The value of column c = h * value_dim + d of a token:
//   x = o[t, h, d] (+ skip[h] * u[t, c]);   with a key sum: x / (max(|o[t, h, value_dim]|, floor[t, h]) + 1e-6)
//   x *= silu(before[t, c]);   x / rms over its group of columns * weight[c % weight_count];
//   x *= sigmoid(behind[t, c])
// Every piece but the norm is optional.  LANES threads (a wave or a block of four) per (token, group).
struct OutputArgs {
  const float* o;
  int heads, value_dim, ones;
  const float* floor;
  const float* skip;
  const float* u;
  int64_t u_ld;
  const float* before;
  int64_t before_ld;
  const float* weight;
  int weight_count;
  float eps;
  int group;               // columns of a group
  const float* behind;
  int64_t behind_ld;
  int64_t out_ld;
  int tokens;
};

__device__ inline float state_output_value(const OutputArgs& p, int64_t t, int c) {
  const int h = c / p.value_dim;
  const int64_t head_row = (t * p.heads + h) * (p.value_dim + p.ones);
  float x = p.o[head_row + (c - h * p.value_dim)];
  if (p.skip != nullptr) x = fmaf(p.skip[h], p.u[t * p.u_ld + c], x);
  if (p.ones) x /= fmaxf(fabsf(p.o[head_row + p.value_dim]), p.floor[t * p.heads + h]) + 1e-6f;
  if (p.before != nullptr) x *= ms_silu(p.before[t * p.before_ld + c]);
  return x;
}

#define MS_HELD 8
template <typename T, int LANES>
__global__ __launch_bounds__(256) void state_output_kernel(const OutputArgs p, T* __restrict__ out) {
  __shared__ float scratch[16];
  const int groups = p.heads * p.value_dim / p.group;
  const int64_t index = LANES == 64 ? (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6) : (int64_t)blockIdx.x;
  const int lane = threadIdx.x % LANES;
  if (index >= (int64_t)p.tokens * groups) return;     // (whole waves, or the whole block)
  const int64_t t = index / groups;
  const int c0 = (int)(index - t * groups) * p.group;
  float held[MS_HELD], squares = 0.f;
#pragma unroll
  for (int j = 0; j < MS_HELD; ++j) {
    const int d = lane + LANES * j;
    held[j] = d < p.group ? state_output_value(p, t, c0 + d) : 0.f;
    squares = fmaf(held[j], held[j], squares);
  }
  for (int d = lane + LANES * MS_HELD; d < p.group; d += LANES) {
    const float x = state_output_value(p, t, c0 + d);
    squares = fmaf(x, x, squares);
  }
  const float total = LANES == 64 ? wave_sum(squares) : block_sum(squares, scratch);
  const float inv = 1.0f / sqrtf(total / (float)p.group + p.eps);
  auto store = [&](const int d, float x) {
    const int c = c0 + d;
    x *= inv * p.weight[c % p.weight_count];
    if (p.behind != nullptr) x *= ms_sigmoid(p.behind[t * p.behind_ld + c]);
    out[t * p.out_ld + c] = from_float<T>(x);
  };
#pragma unroll
  for (int j = 0; j < MS_HELD; ++j)
    if (lane + LANES * j < p.group) store(lane + LANES * j, held[j]);
  for (int d = lane + LANES * MS_HELD; d < p.group; d += LANES) store(d, state_output_value(p, t, c0 + d));
}

extern "C" int ps_state_output(const float* o, int heads, int value_dim, int ones, const float* floor_in,
                               const float* skip, const float* u, int64_t u_ld, const float* before,
                               int64_t before_ld, const float* weight, int weight_count, float eps,
                               int groups, const float* behind, int64_t behind_ld, void* out,
                               int64_t out_ld, int tokens, int dtype, void* stream) {
  const int columns = heads * value_dim;
  PS_REQUIRE(tokens >= 0 && heads > 0 && value_dim > 0 && groups > 0 && columns % groups == 0 &&
                 weight_count > 0 && eps > 0.f,
             "ps_state_output: bad sizes (%d columns in %d groups)", columns, groups);
  PS_REQUIRE(!ones || floor_in != nullptr, "ps_state_output: a key sum needs the floor of its denominator");
  PS_REQUIRE(skip == nullptr || u != nullptr, "ps_state_output: a skip needs its inputs");
  PS_REQUIRE(dtype == PS_F32 || dtype == PS_BF16, "ps_state_output: unknown dtype %d", dtype);
  if (tokens == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const OutputArgs p = {o, heads, value_dim, ones ? 1 : 0, floor_in, skip, u, u_ld, before, before_ld, weight,
                        weight_count, eps, columns / groups, behind, behind_ld, out_ld, tokens};
  const int64_t units = (int64_t)tokens * groups;
  const bool narrow = p.group <= 64 * MS_HELD;
  const int64_t blocks = narrow ? (units + 3) / 4 : units;
  PS_REQUIRE(blocks < ((int64_t)1 << 31), "ps_state_output: too many blocks");
#define PS_LAUNCH_SO(T)                                                                                   \
  do {                                                                                                    \
    if (narrow)                                                                                           \
      hipLaunchKernelGGL((state_output_kernel<T, 64>), dim3((unsigned)blocks), dim3(256), 0, s, p, (T*)out); \
    else                                                                                                  \
      hipLaunchKernelGGL((state_output_kernel<T, 256>), dim3((unsigned)blocks), dim3(256), 0, s, p, (T*)out); \
  } while (0)
  if (dtype == PS_F32) PS_LAUNCH_SO(float);
  else PS_LAUNCH_SO(bf16_t);
#undef PS_LAUNCH_SO
  PS_CHECK_LAUNCH("ps_state_output");
  return 0;
}
