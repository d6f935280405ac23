// What the kernels of matrix-state recurrences share (matrix_state.hip).
#pragma once

#include "common.h"

// Rules of ps_state_prepare and ps_state_scan.
#define PS_STATE_DECAYED 0
#define PS_STATE_DELTA 1

// A step of the recurrence over the items of a batch.
struct StateStep {
  const float* q;            // [tokens, ..] from the first key head's column on
  int64_t q_ld;
  const float* k;
  int64_t k_ld;
  const float* v;            // from the first head's column on
  int64_t v_ld;
  const float* decay;        // decayed: logarithms [tokens, heads]; delta: factors [tokens, heads * key_dim]
  const float* take;         // [tokens, heads]
  float* state;
  int64_t slot_stride;
  float* out;                // [tokens, heads, value_dim (+ 1 with `ones`)]
  const int* cu_tokens;
  const int* slots;
  int heads, key_share;      // heads that share a key/query head
  int key_dim, value_dim;
  int ones;                  // one more column whose value is one for every token
  float q_scale;
  int aligned;               // slots (records, in chunks) start at multiples of 16 bytes
  int vectors;               // so do every head's queries, keys and values
  // the short convolution's raw inputs, kept for the next step (channels 0: none)
  const float* raw;
  int64_t raw_ld;
  int channels, taps;
  int64_t history;
};

// The slot's last taps - 1 raw inputs of (what it kept, then tokens t0 .. t1 - 1), oldest first; a
// thread's channels are first, first + stride, ...
__device__ inline void state_keep_inputs(const StateStep& p, float* slot, int t0, int t1, int first, int stride) {
  const int count = t1 - t0;
  for (int c = first; c < p.channels; c += stride) {
    float* kept = slot + p.history + c;
    for (int j = 0; j < p.taps - 1; ++j) {
      const int local = count - (p.taps - 1) + j;      // place among this step's tokens
      // (ascending j reads place j + count with count >= 1: never one already written)
      kept[(int64_t)j * p.channels] = local >= 0 ? p.raw[(int64_t)(t0 + local) * p.raw_ld + c]
                                                 : kept[(int64_t)(j + count) * p.channels];
    }
  }
}
