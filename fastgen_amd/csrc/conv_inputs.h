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
// The sum runs over the taps in order, oldest first.  Here K is known: all inputs are asked for before any is used.
template <class TS, int K>
__device__ __forceinline__ void conv_pair_taps(const ConvIn& a, const TS* src, int stride, int t, int c, float (&x)[2]) {
  const int b = a.seq_of_token[t], i = t - a.q_start[b];
  float* tail = a.state + (size_t)a.slot_ids[b] * a.slot_stride + (size_t)c * a.row_len + a.tail_off;
  float u[2][K], w[2][K];
#pragma unroll
  for (int e = 0; e < 2; ++e)
#pragma unroll
    for (int j = 0; j < K; ++j) w[e][j] = a.w[(size_t)(c + e) * K + j];
  if (i >= K - 1) {  // uniform: inputs of this step only
    const TS* row = src + (size_t)(t - (K - 1)) * stride + c;
#pragma unroll
    for (int j = 0; j < K; ++j) {
      u[0][j] = to_f<TS>(row[(size_t)j * stride]);
      u[1][j] = to_f<TS>(row[(size_t)j * stride + 1]);
    }
  } else {
#pragma unroll
    for (int j = 0; j < K; ++j) {
      const int idx = i - (K - 1) + j;
      if (idx >= 0) {
        const TS* row = src + (size_t)(t - i + idx) * stride + c;
        u[0][j] = to_f<TS>(row[0]);
        u[1][j] = to_f<TS>(row[1]);
      } else {
        u[0][j] = tail[K - 1 + idx];
        u[1][j] = tail[a.row_len + K - 1 + idx];
      }
    }
  }
#pragma unroll
  for (int e = 0; e < 2; ++e) {
    x[e] = 0.f;
#pragma unroll
    for (int j = 0; j < K; ++j) x[e] = fmaf(u[e][j], w[e][j], x[e]);
  }
  if (a.move) {  // one token a sequence: the inputs but the oldest are the new tail
#pragma unroll
    for (int j = 1; j < K; ++j) {
      tail[j - 1] = u[0][j];
      tail[a.row_len + j - 1] = u[1][j];
    }
  }
}

template <class TS>
__device__ __forceinline__ void conv_pair(const ConvIn& a, const TS* src, int stride, int t, int c, float (&x)[2]) {
  if (a.taps == 4) return conv_pair_taps<TS, 4>(a, src, stride, t, c, x);  // (taps are uniform)
  if (a.taps == 3) return conv_pair_taps<TS, 3>(a, src, stride, t, c, x);
  const int K = a.taps, b = a.seq_of_token[t], t0 = a.q_start[b], i = t - t0;
  float* tail = a.state + (size_t)a.slot_ids[b] * a.slot_stride + (size_t)c * a.row_len + a.tail_off;
  const float* w = a.w + (size_t)c * K;
  float acc0 = 0.f, acc1 = 0.f, u0 = 0.f, u1 = 0.f;
  for (int j = 0; j < K; ++j) {
    const int idx = i - (K - 1) + j;
    if (idx >= 0) {
      const TS* row = src + (size_t)(t0 + idx) * stride + c;
      u0 = to_f<TS>(row[0]);
      u1 = to_f<TS>(row[1]);
    } else {
      u0 = tail[K - 1 + idx];
      u1 = tail[a.row_len + K - 1 + idx];
    }
    if (a.move && j > 0) {  // (one token a sequence: entry j - 1 has been read)
      tail[j - 1] = u0;
      tail[a.row_len + j - 1] = u1;
    }
    acc0 = fmaf(u0, w[j], acc0);
    acc1 = fmaf(u1, w[K + j], acc1);
  }
  x[0] = acc0;
  x[1] = acc1;
}
