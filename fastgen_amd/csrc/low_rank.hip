// The second halves of projections through a narrow middle: y = act(W2 z + b) for columns z of fp32 rows, several such
// products side by side in one launch (a recurrence's decays and its output gate, say).
//
//   kind 0   y = W2 z + b
//   kind 1   y = -rate[n / per] * softplus(W2 z + b)   (the logarithm of a decay; `per` outputs share a rate)
//
// W2 in bfloat16 meets z rounded to bfloat16 on the matrix cores (v_mfma_f32_16x16x32_bf16); W2 in fp32 meets it as it
// is.  Sums and activations are fp32, the result is fp32.
#include "common.h"

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

#define LR_JOBS 2
struct LowRankJob {
  int col, K;                      // the columns col .. col + K - 1 of a row
  const void* w; int N;            // [N, K]
  float* out; int out_stride;
  const float* bias;               // [N] or null
  int kind; const float* rate; int per;
};
struct LowRankArgs {
  const float* src; int src_stride;
  LowRankJob job[LR_JOBS]; int n_jobs;
  int T;
};

__device__ __forceinline__ float low_rank_act(const LowRankJob& j, int n, float y) {
  if (j.bias) y += j.bias[n];
  if (j.kind == 1) y = -j.rate[n / j.per] * (fmaxf(y, 0.f) + log1pf(expf(-fabsf(y))));
  return y;
}

// softplus with the hardware's exponential and logarithm; where 1 + e would lose e's digits, the logarithm's series
__device__ __forceinline__ float low_rank_softplus(float y) {
  const float e = __expf(-fabsf(y));
  const float series = e * (1.f - e * (0.5f - e * (0.33333333f - 0.25f * e)));
  return fmaxf(y, 0.f) + (e < 0.02f ? series : __logf(1.f + e));
}

// grid (ceil(T / (16 MB)), ceil(most outputs / (64 NB)), jobs), 4 waves.  A wave holds its tokens' z (KS steps of 32) in
// registers and takes NB blocks of 16 outputs; acc[mb][i] = y[token 16 mb + (lane & 15)][output 4 (lane >> 4) + i].
template <int MB, int KS, int NB>
__global__ __launch_bounds__(256) void low_rank_mfma_kernel(const LowRankArgs a) {
  const LowRankJob& j = a.job[blockIdx.z];
  const int lane = threadIdx.x % FG_WAVE, wave = threadIdx.x / FG_WAVE, r16 = lane & 15, g = lane >> 4;
  const int m0 = blockIdx.x * 16 * MB, first = (blockIdx.y * 4 + wave) * 16 * NB;
  if (first >= j.N) return;  // whole waves, no barrier below
  bf16x8 z[MB][KS];
#pragma unroll
  for (int mb = 0; mb < MB; ++mb) {
    const float* row = a.src + (size_t)min(m0 + 16 * mb + r16, a.T - 1) * a.src_stride + j.col;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      const int k = 32 * s + 8 * g;
      float v[8];
      load8<float>(row + (k < j.K ? k : 0), v);
#pragma unroll
      for (int i = 0; i < 8; ++i) z[mb][s][i] = (__bf16)(k < j.K ? v[i] : 0.f);
    }
  }
#pragma unroll
  for (int nb = 0; nb < NB; ++nb) {
    const int n0 = first + 16 * nb;
    if (n0 >= j.N) break;  // uniform in the wave
    const int n = n0 + 4 * g;
    float bias[4], rate[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int c = min(n + i, j.N - 1);
      bias[i] = j.bias ? j.bias[c] : 0.f;
      rate[i] = j.kind == 1 ? j.rate[j.per % 16 == 0 ? n0 / j.per : c / j.per] : 0.f;  // (per is uniform)
    }
    const bf16_t* wrow = (const bf16_t*)j.w + (size_t)min(n0 + r16, j.N - 1) * j.K;
    bf16x8 w[KS];
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      const int k = 32 * s + 8 * g;
      w[s] = *(const bf16x8*)(wrow + (k < j.K ? k : 0));  // (beyond K it meets zeros)
    }
    f32x4 acc[MB];
#pragma unroll
    for (int mb = 0; mb < MB; ++mb) {
      acc[mb] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < KS; ++s) acc[mb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[s], z[mb][s], acc[mb], 0, 0, 0);
    }
#pragma unroll
    for (int mb = 0; mb < MB; ++mb) {
      const int t = m0 + 16 * mb + r16;
      if (t >= a.T) continue;
      float* y = j.out + (size_t)t * j.out_stride + n;
      float v[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        v[i] = acc[mb][i] + bias[i];
        if (j.kind == 1) v[i] = -rate[i] * low_rank_softplus(v[i]);  // uniform
      }
      if (n + 3 < j.N && j.out_stride % 4 == 0 && ((uintptr_t)j.out & 15) == 0) {
        *(float4*)y = make_float4(v[0], v[1], v[2], v[3]);
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (n + i < j.N) y[i] = v[i];
      }
    }
  }
}

// Any size, fp32: grid (T, ceil(most outputs / 256), jobs); the token's z in LDS, a thread an output, k ascending.
#define LR_MAX_K 4096
template <class TW>
__global__ __launch_bounds__(256) void low_rank_kernel(const LowRankArgs a) {
  __shared__ float z[LR_MAX_K];
  const LowRankJob& j = a.job[blockIdx.z];
  const float* row = a.src + (size_t)blockIdx.x * a.src_stride + j.col;
  for (int k = threadIdx.x; k < j.K; k += 256) z[k] = row[k];
  __syncthreads();
  const int n = blockIdx.y * 256 + threadIdx.x;
  if (n >= j.N) return;
  const TW* w = (const TW*)j.w + (size_t)n * j.K;
  float acc = 0.f;
  for (int k = 0; k < j.K; ++k) acc = fmaf(to_f<TW>(w[k]), z[k], acc);
  j.out[(size_t)blockIdx.x * j.out_stride + n] = low_rank_act(j, n, acc);
}

// mfma: bf16 weights, K % 8 == 0 and at most 256, columns and row stride of src in multiples of 8, 16-byte aligned rows
extern "C" int fg_low_rank(const LowRankArgs* args, int w_dtype, int mfma, hipStream_t stream) {
  const LowRankArgs& a = *args;
  if (a.T <= 0) return FG_OK;
  if (!a.src || a.n_jobs < 1 || a.n_jobs > LR_JOBS) return FG_ERR_ARG;
  int n_max = 0, k_max = 0;
  for (int i = 0; i < a.n_jobs; ++i) {
    const LowRankJob& j = a.job[i];
    if (j.K <= 0 || j.N <= 0 || j.col < 0 || j.col + j.K > a.src_stride || !j.w || !j.out || j.out_stride < j.N || j.kind < 0 ||
        j.kind > 1 || (j.kind == 1 && (!j.rate || j.per < 1)) || j.K > LR_MAX_K)
      return FG_ERR_ARG;
    if (mfma && (j.K % 8 || j.col % 8)) return FG_ERR_ARG;
    n_max = j.N > n_max ? j.N : n_max;
    k_max = j.K > k_max ? j.K : k_max;
  }
  if (mfma) {
    if (w_dtype != FG_BF16 || k_max > 256 || a.src_stride % 8) return FG_ERR_ARG;
#define GO(MB, KS, NB)                                                                                    \
  do {                                                                                                    \
    const dim3 grid((a.T + 16 * MB - 1) / (16 * MB), (n_max + 64 * NB - 1) / (64 * NB), a.n_jobs);        \
    if (grid.y > 65535) return FG_ERR_ARG;                                                                \
    low_rank_mfma_kernel<MB, KS, NB><<<grid, 256, 0, stream>>>(a);                                        \
  } while (0)
#define PICK(MB, NB)                   \
  do {                                 \
    if (k_max <= 32) GO(MB, 1, NB);    \
    else if (k_max <= 64) GO(MB, 2, NB);  \
    else if (k_max <= 128) GO(MB, 4, NB); \
    else GO(MB, 8, NB);                \
  } while (0)
    if (a.T <= 16) PICK(1, 1);
    else if (a.T <= 256) PICK(2, 1);
    // (a wave converts its tokens' middles for every 16 NB outputs: more of them where that leaves workgroups enough)
    else if ((long long)((a.T + 63) / 64) * ((n_max + 63) / 64) * a.n_jobs < 2048) PICK(4, 1);
    else PICK(4, 2);
#undef PICK
#undef GO
    return fg_launch_status();
  }
  const dim3 grid(a.T, (n_max + 255) / 256, a.n_jobs);
  if (grid.y > 65535) return FG_ERR_ARG;
  if (w_dtype == FG_F32) low_rank_kernel<float><<<grid, 256, 0, stream>>>(a);
  else if (w_dtype == FG_BF16) low_rank_kernel<bf16_t><<<grid, 256, 0, stream>>>(a);
  else return FG_ERR_ARG;
  return fg_launch_status();
}
