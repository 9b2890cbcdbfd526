// A real-gated linear recurrence per channel (the recurrent block of Griffin), all in fp32:
//
//   r = sigmoid(gr), i = sigmoid(gi)         (logits of a block-diagonal product: gates [T, blocks, 2 n], per block its
//                                             n logits gr, then its n logits gi)
//   log a = -r * decay                       (decay[c] > 0: a constant times softplus of a learned number)
//   S <- a S + sqrt(1 - a^2) i u             (from zero; 1 - a^2 as -expm1(2 log a))
//   out = S * gelu_tanh(y + y_bias) * out_scale
//
// A request's state row holds per channel S and behind it the last K - 1 inputs of the convolution that made u
// ([slots, C, row_len]); a whole pass moves both on.  A thread a channel of one sequence; a run of tokens is loaded
// ahead of the run that is computed.  Long prompts are cut into chunks that are scanned side by side in three passes:
// every chunk from zero (its last S and its sum of log a), the state every chunk starts from (lru_chunk_states:
// over a chunk the decay is exp of that sum), every chunk again from its start with its outputs.
#include "common.h"
#include "conv_inputs.h"

#define LRU_THREADS 64
#define LRU_RUN 4  // tokens whose operands are loaded together

struct LruArgs {
  const void* u; int ldu;                // [T, >= C] activation dtype
  const float* gates; int ldg, block;    // [T, >= 2 C]
  const float* decay;                    // [C]
  const float* y; int ldy; const float* y_bias;
  float out_scale;
  const float* x_raw; int ldx; const float* x_bias; int taps;  // the convolution's input rows (for the tail)
  float* state; int row_len;
  const int* slot_ids; const int* q_start;
  void* out; int ldo, C;
  float* chunk_log; float* chunk_state;  // [n_chunks, C]: a pass over chunks; null: a whole pass
  int pass;                              // 0: whole, 1: chunks' sums, 2: chunks' outputs
};

// exact functions for 32-bit operands, the hardware's exponential for bfloat16
template <class TA> __device__ __forceinline__ float lru_exp(float x);
template <> __device__ __forceinline__ float lru_exp<float>(float x) { return expf(x); }
template <> __device__ __forceinline__ float lru_exp<bf16_t>(float x) { return __expf(x); }
template <class TA> __device__ __forceinline__ float lru_sigmoid(float x);
template <> __device__ __forceinline__ float lru_sigmoid<float>(float x) { return 1.f / (1.f + expf(-x)); }
template <> __device__ __forceinline__ float lru_sigmoid<bf16_t>(float x) { return __builtin_amdgcn_rcpf(1.f + __expf(-x)); }
template <class TA> __device__ __forceinline__ float lru_gelu(float z) {
  return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}
// the tanh form of GELU is z * sigmoid(2 sqrt(2/pi) (z + 0.044715 z^3))
template <> __device__ __forceinline__ float lru_gelu<bf16_t>(float z) {
  return z * lru_sigmoid<bf16_t>(1.5957691216057308f * (z + 0.044715f * z * z * z));
}

__device__ __forceinline__ void lru_move_tail(const LruArgs& a, float* row, int c, int t0, int L) {
  float* tail = row + 1;
  const int keep = a.taps - 1;
  const float xb = a.x_bias ? a.x_bias[c] : 0.f;
  float nt[FG_CONV_MAX_TAPS - 1];
#pragma unroll
  for (int j = 0; j < FG_CONV_MAX_TAPS - 1; ++j) {
    if (j < keep) {
      const int src = L - keep + j;
      nt[j] = src >= 0 ? a.x_raw[(size_t)(t0 + src) * a.ldx + c] + xb : tail[j + L];
    }
  }
#pragma unroll
  for (int j = 0; j < FG_CONV_MAX_TAPS - 1; ++j)
    if (j < keep) tail[j] = nt[j];
}

// grid (ceil(C / 64), sequences or chunks)
template <class TA, int PASS>
__global__ __launch_bounds__(LRU_THREADS) void lru_scan_kernel(const LruArgs a) {
  const int c = blockIdx.x * LRU_THREADS + threadIdx.x, b = blockIdx.y;
  if (c >= a.C) return;
  const int t0 = a.q_start[b], t1 = a.q_start[b + 1];
  float* row = PASS == 0 ? a.state + ((size_t)a.slot_ids[b] * a.C + c) * a.row_len : nullptr;
  float S = PASS == 0 ? row[0] : PASS == 1 ? 0.f : a.chunk_state[(size_t)b * a.C + c];
  const float dec = a.decay[c];
  const float yb = PASS != 1 && a.y_bias ? a.y_bias[c] : 0.f;
  const int g_col = (c / a.block) * 2 * a.block + c % a.block;
  const TA* u = (const TA*)a.u + c;
  const float* gates = a.gates + g_col;
  const float* y = a.y + c;
  TA* out = (TA*)a.out + c;
  float log_sum = 0.f;
  float nu[LRU_RUN], nr[LRU_RUN], ni[LRU_RUN], ny[LRU_RUN];
  auto fetch = [&](int t) {
#pragma unroll
    for (int j = 0; j < LRU_RUN; ++j) {
      const size_t tt = (size_t)min(t + j, t1 - 1);  // (never conditional: beyond the run, its last token again)
      nu[j] = to_f<TA>(u[tt * a.ldu]);
      nr[j] = gates[tt * a.ldg];
      ni[j] = gates[tt * a.ldg + a.block];
      if (PASS != 1) ny[j] = y[tt * a.ldy];
    }
  };
  if (t0 < t1) fetch(t0);
  for (int t = t0; t < t1; t += LRU_RUN) {
    const int n = min(LRU_RUN, t1 - t);
    float av[LRU_RUN], bv[LRU_RUN], gv[LRU_RUN];
#pragma unroll
    for (int j = 0; j < LRU_RUN; ++j) {
      const float la = -lru_sigmoid<TA>(nr[j]) * dec;
      av[j] = lru_exp<TA>(la);
      bv[j] = sqrtf(-expm1f(2.f * la)) * lru_sigmoid<TA>(ni[j]) * nu[j];
      if (PASS == 1 && j < n) log_sum += la;
      if (PASS != 1) gv[j] = lru_gelu<TA>(ny[j] + yb) * a.out_scale;
    }
    if (t + LRU_RUN < t1) fetch(t + LRU_RUN);
#pragma unroll
    for (int j = 0; j < LRU_RUN; ++j) {
      if (j < n) {
        S = av[j] * S + bv[j];
        if (PASS != 1) out[(size_t)(t + j) * a.ldo] = from_f<TA>(S * gv[j]);
      }
    }
  }
  if (PASS == 0) {
    row[0] = S;
    if (a.taps > 1) lru_move_tail(a, row, c, t0, t1 - t0);
  } else if (PASS == 1) {
    a.chunk_state[(size_t)b * a.C + c] = S;
    a.chunk_log[(size_t)b * a.C + c] = log_sum;
  }
}

// chunk_state holds what each chunk adds to a zero state and leaves with the state each chunk starts from, for
// sequence b's chunks seq_chunk[b] .. seq_chunk[b + 1] - 1 in order; the sequence's state row and tail move on.
__global__ __launch_bounds__(LRU_THREADS) void lru_chunk_states_kernel(const LruArgs a, const int* __restrict__ seq_chunk) {
  const int c = blockIdx.x * LRU_THREADS + threadIdx.x, b = blockIdx.y;
  if (c >= a.C) return;
  float* row = a.state + ((size_t)a.slot_ids[b] * a.C + c) * a.row_len;
  float S = row[0];
  const int k0 = seq_chunk[b], k1 = seq_chunk[b + 1];
  for (int k = k0; k < k1; k += 8) {
    float add[8], dec[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const size_t at = (size_t)min(k + j, k1 - 1) * a.C + c;
      add[j] = a.chunk_state[at];
      dec[j] = expf(a.chunk_log[at]);
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      if (k + j < k1) {
        a.chunk_state[(size_t)(k + j) * a.C + c] = S;
        S = dec[j] * S + add[j];
      }
    }
  }
  row[0] = S;
  if (a.taps > 1) lru_move_tail(a, row, c, a.q_start[b], a.q_start[b + 1] - a.q_start[b]);
}

static bool lru_ok(const LruArgs& a, int n) {
  return a.C > 0 && a.block > 0 && a.C % a.block == 0 && a.taps >= 1 && a.taps <= FG_CONV_MAX_TAPS && n <= 65535 &&
         a.row_len >= a.taps && a.u && a.gates && a.decay && a.y && a.state && a.out && a.q_start && a.slot_ids &&
         (a.taps == 1 || a.x_raw);
}

// n: sequences (pass 0) or chunks (passes 1 and 2; q_start then holds the chunks' first tokens)
extern "C" int fg_lru_scan(const LruArgs* args, int n, int act_dtype, hipStream_t stream) {
  if (n <= 0) return FG_OK;
  const LruArgs& a = *args;
  if (!lru_ok(a, n) || a.pass < 0 || a.pass > 2 || (a.pass && (!a.chunk_log || !a.chunk_state))) return FG_ERR_ARG;
  const dim3 grid((a.C + LRU_THREADS - 1) / LRU_THREADS, n);
#define GO(TA)                                                                            \
  do {                                                                                    \
    if (a.pass == 0) lru_scan_kernel<TA, 0><<<grid, LRU_THREADS, 0, stream>>>(a);         \
    else if (a.pass == 1) lru_scan_kernel<TA, 1><<<grid, LRU_THREADS, 0, stream>>>(a);    \
    else lru_scan_kernel<TA, 2><<<grid, LRU_THREADS, 0, stream>>>(a);                     \
  } while (0)
  if (act_dtype == FG_F32) GO(float);
  else if (act_dtype == FG_BF16) GO(bf16_t);
  else return FG_ERR_ARG;
#undef GO
  return fg_launch_status();
}

extern "C" int fg_lru_chunk_states(const LruArgs* args, const int* seq_chunk, int n_seqs, hipStream_t stream) {
  if (n_seqs <= 0) return FG_OK;
  const LruArgs& a = *args;
  if (!lru_ok(a, n_seqs) || !a.chunk_log || !a.chunk_state || !seq_chunk) return FG_ERR_ARG;
  lru_chunk_states_kernel<<<dim3((a.C + LRU_THREADS - 1) / LRU_THREADS, n_seqs), LRU_THREADS, 0, stream>>>(a, seq_chunk);
  return fg_launch_status();
}
