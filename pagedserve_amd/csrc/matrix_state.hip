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
// A wave per unit of TT tokens.  Units of the convolution: the first `unit_heads` runs of `head`
// channels each, whose activated values are made unit vectors (the first `scale_heads` of them are
// also multiplied by q_scale), then runs of 64 NR of the other channels.  Then units of 64 NR decays.
struct PrepareArgs {
  const float* proj;
  int64_t ld;
  int col, channels, taps;
  const float* w;          // [taps, channels], the last row is the current token's
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
  int conv_units, decay_units, tokens;
};

template <int NR, int TT>
__global__ __launch_bounds__(256) void state_prepare_kernel(const PrepareArgs p) {
  const int t0 = blockIdx.x * TT;
  const int many = p.tokens - t0 < TT ? p.tokens - t0 : TT;
  const int lane = threadIdx.x & 63;
  const int unit = blockIdx.y * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  if (unit >= p.conv_units + p.decay_units) return;
  if (unit >= p.conv_units) {
    const int first = (unit - p.conv_units) * 64 * NR;
    const int count = p.rule == PS_STATE_DELTA ? p.heads * p.per_head : p.heads;
    for (int tt = 0; tt < many; ++tt) {
      const int64_t t = t0 + tt;
      const float* row = p.proj + t * p.ld;
#pragma unroll
      for (int j = 0; j < NR; ++j) {
        const int c = first + j * 64 + lane;
        if (c < p.heads) {
          const float raw = row[p.take_col + c];
          if (p.rule == PS_STATE_DELTA) {
            p.take[t * p.heads + c] = ms_sigmoid(raw);
          } else {
            const float dt = ms_softplus(raw + p.z_bias[c]);
            p.take[t * p.heads + c] = dt;
            p.decay[t * p.heads + c] = -expf(p.a_log[c]) * dt;
          }
        }
        if (p.rule == PS_STATE_DELTA && c < count) {
          const float step = ms_softplus(p.z[t * p.z_ld + c] + p.z_bias[c]);
          p.decay[t * count + c] = expf(-expf(p.a_log[c / p.per_head]) * step);
        }
      }
    }
    return;
  }
  const bool normed = unit < p.unit_heads;
  const int c0 = normed ? unit * p.head : p.unit_heads * p.head + (unit - p.unit_heads) * 64 * NR;
  const int most = normed ? p.head : 64 * NR;
  const int count = p.channels - c0 < most ? p.channels - c0 : most;
  const int item = p.tok_item[t0];
  const int first = p.cu_tokens[item];
  float value[TT][NR];
  // every load below is unconditional, from the last channel where a lane has none
  if (TT > 1 && many == TT && p.taps <= 4 && t0 - first >= p.taps - 1 && t0 + TT <= p.cu_tokens[item + 1]) {
    // all inputs are of this step and this item: each is loaded once for the tokens that see it
#pragma unroll
    for (int j = 0; j < NR; ++j) {
      const int c = c0 + (j * 64 + lane < count ? j * 64 + lane : count - 1);
      float x[TT + 3], w[4];
#pragma unroll
      for (int i = 0; i < TT + 3; ++i) {
        const int t = t0 - 3 + i > 0 ? t0 - 3 + i : 0;
        x[i] = p.proj[(int64_t)t * p.ld + p.col + c];
      }
#pragma unroll
      for (int back = 0; back < 4; ++back)
        w[back] = back < p.taps ? p.w[(int64_t)(p.taps - 1 - back) * p.channels + c] : 0.f;
      const float start = p.bias ? p.bias[c] : 0.f;
#pragma unroll
      for (int tt = 0; tt < TT; ++tt) {
        float sum = start;
#pragma unroll
        for (int back = 3; back >= 0; --back) sum = back < p.taps ? fmaf(w[back], x[tt + 3 - back], sum) : sum;
        value[tt][j] = ms_silu(sum);
      }
    }
  } else {
#pragma unroll
    for (int tt = 0; tt < TT; ++tt) {
      const int t = tt < many ? t0 + tt : t0;
      const int it = TT > 1 ? p.tok_item[t] : item;
      const int begin = TT > 1 ? p.cu_tokens[it] : first;
      const float* kept = p.state + p.slots[it] * p.slot_stride + p.history;
      const float* row = p.proj + (int64_t)t * p.ld + p.col;
      float sum[NR];
#pragma unroll
      for (int j = 0; j < NR; ++j)
        sum[j] = p.bias ? p.bias[c0 + (j * 64 + lane < count ? j * 64 + lane : count - 1)] : 0.f;
      for (int tap0 = 0; tap0 < p.taps; tap0 += 4) {
        float x[4][NR], w[4][NR];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int tap = tap0 + i < p.taps ? tap0 + i : p.taps - 1;
          const int back = p.taps - 1 - tap;          // the input `back` tokens before this one
          const int local = (t - begin) - back;       // its place among the item's tokens of this step
          const float* from = local >= 0 ? row - (int64_t)back * p.ld
                                         : kept + (int64_t)(p.taps - 1 + local) * p.channels;
#pragma unroll
          for (int j = 0; j < NR; ++j) {
            const int c = c0 + (j * 64 + lane < count ? j * 64 + lane : count - 1);
            x[i][j] = from[c];
            w[i][j] = p.w[(int64_t)tap * p.channels + c];
          }
        }
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
          for (int j = 0; j < NR; ++j)
            if (tap0 + i < p.taps) sum[j] = fmaf(w[i][j], x[i][j], sum[j]);
      }
#pragma unroll
      for (int j = 0; j < NR; ++j) value[tt][j] = ms_silu(sum[j]);
    }
  }
#pragma unroll
  for (int tt = 0; tt < TT; ++tt) {
    if (tt >= many) break;
    float factor = 1.f;
    if (normed) {
      float squares = 0.f;
#pragma unroll
      for (int j = 0; j < NR; ++j) {
        const float v = j * 64 + lane < count ? value[tt][j] : 0.f;
        squares = fmaf(v, v, squares);
      }
      factor = 1.0f / sqrtf(wave_sum(squares) + 1e-6f);
      if (unit < p.scale_heads) factor *= p.q_scale;
    }
#pragma unroll
    for (int j = 0; j < NR; ++j) {
      const int d = j * 64 + lane;
      if (d < count) p.out[(int64_t)(t0 + tt) * p.channels + c0 + d] = value[tt][j] * factor;
    }
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
                 (unit_heads == 0 || (head > 0 && head <= 256)),
             "ps_state_prepare: %d heads of %d do not fit %d channels (heads of up to 256)", unit_heads, head,
             channels);
  PS_REQUIRE(rule == PS_STATE_DECAYED || (rule == PS_STATE_DELTA && z != nullptr),
             "ps_state_prepare: rule %d", rule);
  if (tokens == 0) return 0;
  PrepareArgs p = {proj, ld, col, channels, taps, w, bias, state, slot_stride, history, out, unit_heads,
                   head, scale_heads, q_scale, rule, heads, per_head, z, z_ld, z_bias, a_log, take_col,
                   decay, take, tok_item, cu_tokens, slots, 0, 0, tokens};
  // few tokens: as many waves as there are runs of 64 channels; many: several tokens to a wave, which
  // share their inputs
  const bool few = tokens <= 64;
  const int nr = unit_heads > 0 ? (head <= 64 ? 1 : (head <= 128 ? 2 : 4)) : (few ? 1 : 2);
  p.conv_units = unit_heads + (channels - unit_heads * head + 64 * nr - 1) / (64 * nr);
  const int decays = rule == PS_STATE_DELTA ? heads * per_head : heads;
  p.decay_units = (decays + 64 * nr - 1) / (64 * nr);
  const int units = p.conv_units + p.decay_units;
  PS_REQUIRE((units + 3) / 4 <= 65535, "ps_state_prepare: too many channels");
#define PS_LAUNCH_PREP(NR, TT)                                                                          \
  hipLaunchKernelGGL((state_prepare_kernel<NR, TT>), dim3((tokens + TT - 1) / TT, (units + 3) / 4),     \
                     dim3(256), 0, (hipStream_t)stream, p)
#define PS_LAUNCH_PREP_T(NR)              \
  do {                                    \
    if (few) PS_LAUNCH_PREP(NR, 1);       \
    else PS_LAUNCH_PREP(NR, 8);           \
  } while (0)
  if (nr == 1) PS_LAUNCH_PREP_T(1);
  else if (nr == 2) PS_LAUNCH_PREP_T(2);
  else PS_LAUNCH_PREP_T(4);
#undef PS_LAUNCH_PREP_T
#undef PS_LAUNCH_PREP
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
// CHUNK tokens wait in LDS for all four waves; the next chunk's loads travel while this one is
// worked on.  The chain from token to token is what bounds a long portion, and one wave has a SIMD to
// itself, so nothing may stand between two tokens: a chunk's tokens are one straight run of
// instructions (places behind the item's last token decay by one and add nothing), and the lanes'
// shares of the outputs stay in registers until they are summed for GROUPS tokens at once.

// values[i] of every lane of an aligned group of N = the share of token i; returns the sum over the
// group's lanes of token (lane % N).  Every step halves the tokens a lane still cares for.
template <int N>
__device__ inline float sum_transposed(float (&values)[N], int lane) {
  float v[N];
#pragma unroll
  for (int i = 0; i < N; ++i) v[i] = values[i];
  // a lane keeps the tokens whose bit is its own and takes its partner's share of them (the partner: the
  // mirrored lane of 16 or 8, then the lane with that bit turned)
  auto halve = [&](auto exchange, const int half) {
    const bool upper = (lane & half) != 0;
#pragma unroll
    for (int i = 0; i < N / 2; ++i) {
      if (i < half) {
        const float keep = upper ? v[i + half] : v[i];
        const float give = upper ? v[i] : v[i + half];
        v[i] = keep + exchange(give);
      }
    }
  };
  if constexpr (N >= 16) halve([](float x) { return lane_exchange<0x140>(x); }, 8);
  if constexpr (N >= 8) halve([](float x) { return lane_exchange<0x141>(x); }, 4);
  if constexpr (N >= 4) halve([](float x) { return lane_exchange<0x4E>(x); }, 2);
  halve([](float x) { return lane_exchange<0xB1>(x); }, 1);
  return v[0];
}

template <int RPL, int GROUPS, int CHUNK, bool DELTA>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(1, 2))) void state_walk_kernel(const StateStep p) {
  constexpr int COLS = 64 / GROUPS;                // columns of a wave
  constexpr int BLOCK_COLS = 4 * COLS;
  constexpr int ROWS = GROUPS * RPL;               // key rows with padding up to the lanes' share
  constexpr int PAD = RPL < 4 ? 4 : RPL + 4;       // row groups start in different banks
  constexpr int PER = (CHUNK * ROWS + 255) / 256;  // values of a chunk per thread and array
  constexpr int PER_V = (CHUNK * BLOCK_COLS + 255) / 256;
  constexpr int RUN = CHUNK < GROUPS ? CHUNK : GROUPS;   // tokens whose outputs are summed together
  static_assert(CHUNK == 1 || CHUNK % GROUPS == 0, "whole runs of tokens, or one token");
  __shared__ __attribute__((aligned(16))) float s_q[CHUNK][GROUPS * PAD];
  __shared__ __attribute__((aligned(16))) float s_k[CHUNK][GROUPS * PAD];
  __shared__ __attribute__((aligned(16))) float s_a[DELTA ? CHUNK : 1][GROUPS * PAD];
  __shared__ float s_v[CHUNK][BLOCK_COLS];
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
  // a chunk on its way from memory; two of them travel at a time (a chunk's work is shorter than a trip)
  struct Coming {
    float q[PER], k[PER], a[DELTA ? PER : 1], v[PER_V], d, w;
  };
  Coming even, odd;
  // A thread's places within a chunk are the same in every chunk: their distances from the chunk's first
  // row are worked out once, and a chunk's loads are a scalar address and such a distance each.
  int place_tt[PER], place_at[PER], off_q[PER], off_k[PER], off_a[DELTA ? PER : 1], col_q[PER];
  bool place_row[PER];
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    const int idx = tid + j * 256;
    const int tt = idx / ROWS;
    const int r = idx - tt * ROWS;
    place_tt[j] = tt;
    place_at[j] = tt * (GROUPS * PAD) + (r / RPL) * PAD + (r % RPL);
    place_row[j] = r < p.key_dim;
    col_q[j] = r < p.key_dim ? r : 0;
    off_q[j] = tt * (int)p.q_ld + col_q[j];
    off_k[j] = tt * (int)p.k_ld + col_q[j];
    if (DELTA) off_a[j] = tt * (int)a_ld + col_q[j];
  }
  int v_tt[PER_V], v_at[PER_V], off_v[PER_V];
  float v_factor[PER_V], v_add[PER_V];
#pragma unroll
  for (int j = 0; j < PER_V; ++j) {
    const int idx = tid + j * 256;
    v_tt[j] = idx / BLOCK_COLS;
    const int c = col0 + (idx - v_tt[j] * BLOCK_COLS);
    v_at[j] = c < p.value_dim ? c : 0;
    off_v[j] = v_tt[j] * (int)p.v_ld + v_at[j];
    // (the column behind the values sums the keys alone: its value is one)
    v_factor[j] = c < p.value_dim ? 1.f : 0.f;
    v_add[j] = p.ones && c == p.value_dim ? 1.f : 0.f;
  }
  // every load is unconditional (from the chunk's first row where the item has no such token); what lies
  // outside is masked when stored
  auto fetch = [&](Coming& in, const int base) {
    if (base >= t1) return;
    const int count = (t1 - base) < CHUNK ? (t1 - base) : CHUNK;
    const float* q_row = q_base + (int64_t)base * p.q_ld;
    const float* k_row = k_base + (int64_t)base * p.k_ld;
    const float* a_row = DELTA ? a_base + (int64_t)base * a_ld : nullptr;
    const float* v_row = v_base + (int64_t)base * p.v_ld;
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const bool there = place_tt[j] < count;
      in.q[j] = q_row[there ? off_q[j] : col_q[j]];
      in.k[j] = k_row[there ? off_k[j] : col_q[j]];
      if (DELTA) in.a[j] = a_row[there ? off_a[j] : col_q[j]];
    }
#pragma unroll
    for (int j = 0; j < PER_V; ++j) in.v[j] = v_row[v_tt[j] < count ? off_v[j] : v_at[j]];
    if (tid < CHUNK) {
      const int64_t at = (int64_t)(base + (tid < count ? tid : 0)) * p.heads + head;
      in.w = p.take[at];
      if (!DELTA) in.d = p.decay[at];
    }
  };
  auto stash = [&](const Coming& in, const int base) {
    const int count = (t1 - base) < CHUNK ? (t1 - base) : CHUNK;
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const bool valid = place_tt[j] < count && place_row[j];
      if (CHUNK * ROWS % 256 == 0 || place_tt[j] < CHUNK) {
        (&s_q[0][0])[place_at[j]] = valid ? in.q[j] * p.q_scale : 0.f;
        (&s_k[0][0])[place_at[j]] = valid ? in.k[j] : 0.f;
        if (DELTA) (&s_a[0][0])[place_at[j]] = valid ? in.a[j] : 1.f;
      }
    }
#pragma unroll
    for (int j = 0; j < PER_V; ++j)
      if (CHUNK * BLOCK_COLS % 256 == 0 || v_tt[j] < CHUNK)
        (&s_v[0][0])[tid + j * 256] = v_tt[j] < count ? fmaf(in.v[j], v_factor[j], v_add[j]) : 0.f;
    if (tid < CHUNK) {
      s_w[tid] = tid < count ? in.w : 0.f;
      s_d[tid] = DELTA || tid >= count ? 1.f : expf(in.d);
    }
  };
  fetch(even, t0);
  fetch(odd, t0 + CHUNK);
  float S[RPL];
  const int rows_mine = p.key_dim - group * RPL;   // key rows from the lane's first on
  const bool whole = RPL % 4 == 0 && p.key_dim % 4 == 0 && p.aligned;
  if (whole) {
#pragma unroll
    for (int i = 0; i < RPL; i += 4) {
      float4 four = make_float4(0.f, 0.f, 0.f, 0.f);
      if (i < rows_mine && has_col) four = *reinterpret_cast<const float4*>(s_ptr + i);
      S[i] = four.x;
      S[(i + 1) % RPL] = four.y;
      S[(i + 2) % RPL] = four.z;
      S[(i + 3) % RPL] = four.w;
    }
  } else {
#pragma unroll
    for (int i = 0; i < RPL; ++i) S[i] = (i < rows_mine && has_col) ? s_ptr[i] : 0.f;
  }
  const int out_ld = p.heads * columns;
  auto work = [&](Coming& in, const int base) {
    __syncthreads();      // the chunk before has been read
    stash(in, base);
    __syncthreads();
    fetch(in, base + 2 * CHUNK);
    // what a token's step reads from LDS, into registers
    struct Operands {
      float q[RPL], k[RPL], a[DELTA ? RPL : 1], v, w, d;
    };
    auto load = [&](const int tt, Operands& in) {
#pragma unroll
      for (int i = 0; i < RPL; i += 4) {
        *reinterpret_cast<float4*>(&in.k[i]) = *reinterpret_cast<const float4*>(&s_k[tt][group * PAD + i]);
        if (DELTA)
          *reinterpret_cast<float4*>(&in.a[i % (DELTA ? RPL : 1)]) = *reinterpret_cast<const float4*>(&s_a[tt][group * PAD + i]);
        *reinterpret_cast<float4*>(&in.q[i]) = *reinterpret_cast<const float4*>(&s_q[tt][group * PAD + i]);
      }
      in.v = s_v[tt][mine];
      in.w = s_w[tt];
      in.d = DELTA ? 1.f : s_d[tt];
    };
    // the lane's share of a token's output
    auto token = [&](const Operands& in) -> float {
      float v = in.v;
      if (DELTA) {
        float dot0 = 0.f, dot1 = 0.f;
#pragma unroll
        for (int i = 0; i < RPL; ++i) {
          S[i] *= in.a[i % (DELTA ? RPL : 1)];
          if (i & 1) dot1 = fmaf(S[i], in.k[i], dot1);
          else dot0 = fmaf(S[i], in.k[i], dot0);
        }
        v = in.w * (v - lanes_sum<GROUPS>(dot0 + dot1));
      } else {
        v *= in.w;
#pragma unroll
        for (int i = 0; i < RPL; ++i) S[i] *= in.d;
      }
      float o0 = 0.f, o1 = 0.f;
#pragma unroll
      for (int i = 0; i < RPL; ++i) {
        S[i] = fmaf(in.k[i], v, S[i]);
        if (i & 1) o1 = fmaf(S[i], in.q[i], o1);
        else o0 = fmaf(S[i], in.q[i], o0);
      }
      return o0 + o1;
    };
    if constexpr (CHUNK == 1) {
      Operands in;
      load(0, in);
      const float o = lanes_sum<GROUPS>(token(in));
      if (group == 0 && has_col) p.out[((int64_t)base * p.heads + head) * columns + col] = o;
    } else {
      // the reads of the next tokens are on their way while a token is worked on: the barriers keep the
      // compiler from moving them down to where they are used
      constexpr int AHEAD = RPL > 8 ? 1 : 2;
      Operands in[AHEAD + 1];
#pragma unroll
      for (int i = 0; i < AHEAD; ++i) load(i, in[i]);
#pragma unroll
      for (int run = 0; run < CHUNK; run += RUN) {
        float shares[GROUPS];
#pragma unroll
        for (int i = 0; i < GROUPS; ++i) {
          const int tt = run + i;
          if (tt + AHEAD < CHUNK) load(tt + AHEAD, in[(tt + AHEAD) % (AHEAD + 1)]);
          __builtin_amdgcn_sched_barrier(0);
          shares[i] = token(in[tt % (AHEAD + 1)]);
          __builtin_amdgcn_sched_barrier(0);
        }
        const float o = sum_transposed<GROUPS>(shares, lane);
        if (base + run + group < t1 && has_col)
          (p.out + (int64_t)(base + run) * out_ld + head * columns)[group * out_ld + col] = o;
      }
    }
  };
  for (int base = t0; base < t1; base += 2 * CHUNK) {
    work(even, base);
    if (base + CHUNK < t1) work(odd, base + CHUNK);
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
                       heads, key_share, key_dim, value_dim, ones, q_scale, aligned, 0, raw, raw_ld, channels, taps,
                       history};
  const bool brief = longest == 1;
#define PS_LAUNCH_WALK_D(RPL, GROUPS, CHUNK, DELTA)                                               \
  hipLaunchKernelGGL((state_walk_kernel<RPL, GROUPS, CHUNK, DELTA>),                              \
                     dim3(items, heads, (columns + 256 / GROUPS - 1) / (256 / GROUPS)), dim3(256), 0, s, p)
#define PS_LAUNCH_WALK(RPL, GROUPS, CHUNK)                  \
  do {                                                      \
    if (rule == PS_STATE_DELTA) {                           \
      if (brief) PS_LAUNCH_WALK_D(RPL, GROUPS, 1, true);    \
      else PS_LAUNCH_WALK_D(RPL, GROUPS, CHUNK, true);      \
    } else {                                                \
      if (brief) PS_LAUNCH_WALK_D(RPL, GROUPS, 1, false);   \
      else PS_LAUNCH_WALK_D(RPL, GROUPS, CHUNK, false);     \
    }                                                       \
  } while (0)
  if (key_dim <= 16) PS_LAUNCH_WALK(4, 4, 16);
  else if (key_dim <= 32) PS_LAUNCH_WALK(4, 8, 16);
  else if (key_dim <= 64) PS_LAUNCH_WALK(4, 16, 16);
  else if (key_dim <= 128) PS_LAUNCH_WALK(8, 16, 16);
  else PS_LAUNCH_WALK(16, 16, 16);
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

// A thread's share of its group: HELD columns, every load of which leaves before any is used (from the
// group's last column where a thread has none).
template <typename T, int LANES, int HELD>
__global__ __launch_bounds__(256) void state_output_kernel(const OutputArgs p, T* __restrict__ out) {
  __shared__ float scratch[16];
  const int groups = p.heads * p.value_dim / p.group;
  const int64_t index = LANES == 64 ? (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6) : (int64_t)blockIdx.x;
  const int lane = threadIdx.x % LANES;
  if (index >= (int64_t)p.tokens * groups) return;     // (whole waves, or the whole block)
  const int64_t t = index / groups;
  const int c0 = (int)(index - t * groups) * p.group;
  const float per_head = 1.0f / (float)p.value_dim;
  const bool shared_weight = p.weight_count == p.value_dim;
  float x[HELD], u[HELD], skip[HELD], sum[HELD], floor_of[HELD], before[HELD], behind[HELD], weight[HELD];
#pragma unroll
  for (int j = 0; j < HELD; ++j) {
    const int d = lane + LANES * j;
    const int c = c0 + (d < p.group ? d : p.group - 1);
    const int h = (int)(((float)c + 0.5f) * per_head);   // c / value_dim (columns are far fewer than 2^20)
    const int64_t row = (t * p.heads + h) * (p.value_dim + p.ones);
    x[j] = p.o[row + (c - h * p.value_dim)];
    weight[j] = p.weight[shared_weight ? c - h * p.value_dim : c];
    u[j] = skip[j] = before[j] = behind[j] = 0.f;
    sum[j] = floor_of[j] = 1.f;
    if (p.skip != nullptr) {
      u[j] = p.u[t * p.u_ld + c];
      skip[j] = p.skip[h];
    }
    if (p.ones) {
      sum[j] = p.o[row + p.value_dim];
      floor_of[j] = p.floor[t * p.heads + h];
    }
    if (p.before != nullptr) before[j] = p.before[t * p.before_ld + c];
    if (p.behind != nullptr) behind[j] = p.behind[t * p.behind_ld + c];
  }
  float squares = 0.f;
#pragma unroll
  for (int j = 0; j < HELD; ++j) {
    x[j] = fmaf(skip[j], u[j], x[j]);
    if (p.ones) x[j] /= fmaxf(fabsf(sum[j]), floor_of[j]) + 1e-6f;
    if (p.before != nullptr) x[j] *= ms_silu(before[j]);
    if (lane + LANES * j < p.group) squares = fmaf(x[j], x[j], squares);
  }
  const float total = LANES == 64 ? wave_sum(squares) : block_sum(squares, scratch);
  const float inv = 1.0f / sqrtf(total / (float)p.group + p.eps);
#pragma unroll
  for (int j = 0; j < HELD; ++j) {
    const int d = lane + LANES * j;
    if (d < p.group) {
      float v = x[j] * (inv * weight[j]);
      if (p.behind != nullptr) v *= ms_sigmoid(behind[j]);
      out[t * p.out_ld + c0 + d] = from_float<T>(v);
    }
  }
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
  const bool narrow = p.group <= 256;
  const int held = (p.group + (narrow ? 63 : 255)) / (narrow ? 64 : 256);
  PS_REQUIRE(held <= 32, "ps_state_output: groups of %d columns, at most 8192", p.group);
  const int64_t blocks = narrow ? (units + 3) / 4 : units;
  PS_REQUIRE(blocks < ((int64_t)1 << 31), "ps_state_output: too many blocks");
#define PS_LAUNCH_SO(T, LANES, HELD) \
  hipLaunchKernelGGL((state_output_kernel<T, LANES, HELD>), dim3((unsigned)blocks), dim3(256), 0, s, p, (T*)out)
#define PS_LAUNCH_SO_T(T)                               \
  do {                                                  \
    if (narrow && held == 1) PS_LAUNCH_SO(T, 64, 1);    \
    else if (narrow && held == 2) PS_LAUNCH_SO(T, 64, 2); \
    else if (narrow) PS_LAUNCH_SO(T, 64, 4);            \
    else if (held <= 2) PS_LAUNCH_SO(T, 256, 2);        \
    else if (held <= 4) PS_LAUNCH_SO(T, 256, 4);        \
    else if (held <= 8) PS_LAUNCH_SO(T, 256, 8);        \
    else PS_LAUNCH_SO(T, 256, 32);                      \
  } while (0)
  if (dtype == PS_F32) PS_LAUNCH_SO_T(float);
  else PS_LAUNCH_SO_T(bf16_t);
#undef PS_LAUNCH_SO_T
#undef PS_LAUNCH_SO
  PS_CHECK_LAUNCH("ps_state_output");
  return 0;
}
