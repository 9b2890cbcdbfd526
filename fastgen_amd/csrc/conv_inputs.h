// A short causal convolution per channel that a kernel applies where it reads its rows: the last tap meets the
// token itself, and inputs of earlier steps come from a state row per request, channel c's K - 1 values (oldest
// first) at state + slot * slot_stride + c * row_len + tail_off.
#pragma once
#include "common.h"

#define FG_CONV_MAX_TAPS 16

struct ConvIn {
  const float* w; int taps;          // [C, K]; null: no convolution
  float* state; long long slot_stride; int channels, row_len, tail_off;
  const int* slot_ids; const int* seq_of_token; const int* q_start;
  int move;                          // every sequence brings one token: its tail is moved on here
};

static inline bool fg_conv_ok(const ConvIn& c) {
  return c.taps >= 1 && c.taps <= FG_CONV_MAX_TAPS && c.state && c.tail_off >= 0 && c.row_len >= c.tail_off + c.taps - 1 &&
         c.channels > 0 && c.slot_stride >= 0 && c.slot_ids && c.seq_of_token && c.q_start;
}

// Channels c and c + 1 of token t, from the rows src [T, stride] (channel = column); with `move` also their tails.
template <class TS>
__device__ __forceinline__ void conv_pair(const ConvIn& a, const TS* src, int stride, int t, int c, float (&x)[2]) {
  const int K = a.taps, b = a.seq_of_token[t], t0 = a.q_start[b], i = t - t0;
  float* tail = a.state + (size_t)a.slot_ids[b] * a.slot_stride + (size_t)c * a.row_len + a.tail_off;
  const float* w = a.w + (size_t)c * K;
  float acc0 = 0.f, acc1 = 0.f;
  for (int j = 0; j < K; ++j) {
    const int idx = i - (K - 1) + j;
    float u0, u1;
    if (idx >= 0) {
      const TS* row = src + (size_t)(t0 + idx) * stride + c;
      u0 = to_f<TS>(row[0]);
      u1 = to_f<TS>(row[1]);
    } else {
      u0 = tail[K - 1 + idx];
      u1 = tail[a.row_len + K - 1 + idx];
    }
    acc0 = fmaf(u0, w[j], acc0);
    acc1 = fmaf(u1, w[K + j], acc1);
  }
  if (a.move && K > 1) {
    for (int j = 0; j + 2 < K; ++j) {
      tail[j] = tail[j + 1];
      tail[a.row_len + j] = tail[a.row_len + j + 1];
    }
    const TS* row = src + (size_t)t * stride + c;
    tail[K - 2] = to_f<TS>(row[0]);
    tail[a.row_len + K - 2] = to_f<TS>(row[1]);
  }
  x[0] = acc0;
  x[1] = acc1;
}
