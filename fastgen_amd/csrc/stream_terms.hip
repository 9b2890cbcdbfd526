// What several sublayers leave to be added to the residual stream, added and normed in one pass.
//
//   h += sum_j s_j (.) n_j(x_j + b_j)      up to three terms, in their order
//   h += again                             rows that enter the stream once more (or none)
//   out_k = h / rms(h) * w_k               up to two norms of the same row (they share its root mean square)
//
// x_j is a row of the activation dtype or the sum, in order, of fp32 partial results of a product whose k range was
// cut; b_j a bias per channel or none; n_j the division by the row's root mean square or nothing; s_j a vector per channel
// (a norm's weight, a learned scale, constants: their product) or none.  All fp32, one rounding at the store of out.  With
// `rows` only the gathered rows are computed and h is left as it was.  A workgroup a row, which it keeps in registers.
#include "common.h"

#define TM_THREADS 256
#define TM_TERMS 3
#define TM_MAX_DIM 16384

struct StreamTerm {
  const void* rows;                         // [T, dim], or null
  const float* parts; int n_parts; long long part_stride;  // fp32 [n_parts, T, dim], or null
  const float* bias; const float* scale;    // [dim] or null
  int normed; float eps;
};
struct StreamTermsArgs {
  float* h;
  StreamTerm term[TM_TERMS]; int n_terms;
  const float* again;                       // fp32 [T, dim] or null
  const void* w[2]; void* out[2];           // null: no such norm
  const int* rows;
  int dim; float eps;
};

template <int VEC, class T> __device__ __forceinline__ void tm_load(const T* p, float (&v)[VEC]) {
  if constexpr (VEC == 8) load8<T>(p, v);
  else v[0] = to_f<T>(p[0]);
}
template <int VEC, class T> __device__ __forceinline__ void tm_store(T* p, const float (&v)[VEC]) {
  if constexpr (VEC == 8) store8<T>(p, v);
  else p[0] = from_f<T>(v[0]);
}

// NIT groups of VEC elements a thread.  Loads are never conditional on the group: one beyond the row reads the row's last
// VEC elements and counts for nothing.
template <class TA, class TW, int VEC, int NIT>
__global__ __launch_bounds__(TM_THREADS) void stream_terms_kernel(const StreamTermsArgs a) {
  __shared__ float red[TM_TERMS + 1][16];
  const int r = blockIdx.x, dim = a.dim;
  const size_t src = a.rows ? (size_t)a.rows[r] : (size_t)r;
  float* hrow = a.h + src * dim;
  int e[NIT], ec[NIT];
#pragma unroll
  for (int it = 0; it < NIT; ++it) {
    e[it] = (threadIdx.x + it * TM_THREADS) * VEC;
    ec[it] = min(e[it], dim - VEC);
  }
  float v[NIT][VEC], d[TM_TERMS][NIT][VEC], ss[TM_TERMS];
#pragma unroll
  for (int it = 0; it < NIT; ++it) tm_load<VEC>(hrow + ec[it], v[it]);
  bool any_normed = false;
#pragma unroll
  for (int j = 0; j < TM_TERMS; ++j) {
    ss[j] = 0.f;
    if (j >= a.n_terms) continue;  // uniform
    const StreamTerm& t = a.term[j];
    if (t.rows) {
      const TA* row = (const TA*)t.rows + src * dim;
#pragma unroll
      for (int it = 0; it < NIT; ++it) tm_load<VEC>(row + ec[it], d[j][it]);
    } else {
      const float* row = t.parts + src * dim;
#pragma unroll
      for (int it = 0; it < NIT; ++it) tm_load<VEC>(row + ec[it], d[j][it]);
      constexpr int PB = NIT * VEC <= 16 ? 4 : 1;  // partial results whose loads are in flight together
      for (int p0 = 1; p0 < t.n_parts; p0 += PB) {
        float x[PB][NIT][VEC];
#pragma unroll
        for (int p = 0; p < PB; ++p)
#pragma unroll
          for (int it = 0; it < NIT; ++it) tm_load<VEC>(row + (size_t)min(p0 + p, t.n_parts - 1) * t.part_stride + ec[it], x[p][it]);
#pragma unroll
        for (int p = 0; p < PB; ++p)
#pragma unroll
          for (int it = 0; it < NIT; ++it)
#pragma unroll
            for (int i = 0; i < VEC; ++i) d[j][it][i] += p0 + p < t.n_parts ? x[p][it][i] : 0.f;
      }
    }
    if (t.bias) {
#pragma unroll
      for (int it = 0; it < NIT; ++it) {
        float b[VEC];
        tm_load<VEC>(t.bias + ec[it], b);
#pragma unroll
        for (int i = 0; i < VEC; ++i) d[j][it][i] += b[i];
      }
    }
    if (t.normed) {
      any_normed = true;
#pragma unroll
      for (int it = 0; it < NIT; ++it)
        if (e[it] < dim) {
#pragma unroll
          for (int i = 0; i < VEC; ++i) ss[j] += d[j][it][i] * d[j][it][i];
        }
    }
  }
  const int lane = threadIdx.x % FG_WAVE, wave = threadIdx.x / FG_WAVE;
  if (any_normed) {  // uniform: the terms' sums of squares cross the workgroup together
#pragma unroll
    for (int j = 0; j < TM_TERMS; ++j) {
      const float s = wave_sum(ss[j]);
      if (lane == 0) red[j][wave] = s;
    }
    __syncthreads();
#pragma unroll
    for (int j = 0; j < TM_TERMS; ++j) {
      float s = 0.f;
      for (int w = 0; w < TM_THREADS / FG_WAVE; ++w) s += red[j][w];
      ss[j] = s;
    }
  }
#pragma unroll
  for (int j = 0; j < TM_TERMS; ++j) {
    if (j >= a.n_terms) continue;
    const StreamTerm& t = a.term[j];
    const float mul = t.normed ? rsqrtf(ss[j] / (float)dim + t.eps) : 1.f;
#pragma unroll
    for (int it = 0; it < NIT; ++it) {
      float s[VEC];
      if (t.scale) {
        tm_load<VEC>(t.scale + ec[it], s);
      } else {
#pragma unroll
        for (int i = 0; i < VEC; ++i) s[i] = 1.f;
      }
#pragma unroll
      for (int i = 0; i < VEC; ++i) v[it][i] += d[j][it][i] * mul * s[i];
    }
  }
  if (a.again) {
#pragma unroll
    for (int it = 0; it < NIT; ++it) {
      float x[VEC];
      tm_load<VEC>(a.again + src * dim + ec[it], x);
#pragma unroll
      for (int i = 0; i < VEC; ++i) v[it][i] += x[i];
    }
  }
  if (!a.rows && (a.n_terms > 0 || a.again)) {
#pragma unroll
    for (int it = 0; it < NIT; ++it)
      if (e[it] < dim) tm_store<VEC>(hrow + e[it], v[it]);
  }
  if (!a.out[0]) return;  // uniform
  float s2 = 0.f;
#pragma unroll
  for (int it = 0; it < NIT; ++it)
    if (e[it] < dim) {
#pragma unroll
      for (int i = 0; i < VEC; ++i) s2 += v[it][i] * v[it][i];
    }
  s2 = wave_sum(s2);
  if (lane == 0) red[TM_TERMS][wave] = s2;
  __syncthreads();
  s2 = 0.f;
  for (int w = 0; w < TM_THREADS / FG_WAVE; ++w) s2 += red[TM_TERMS][w];
  const float rstd = rsqrtf(s2 / (float)dim + a.eps);
#pragma unroll
  for (int k = 0; k < 2; ++k) {
    if (!a.out[k]) continue;  // uniform
    TA* orow = (TA*)a.out[k] + (size_t)r * dim;
#pragma unroll
    for (int it = 0; it < NIT; ++it) {
      float wv[VEC], o[VEC];
      tm_load<VEC>((const TW*)a.w[k] + ec[it], wv);
#pragma unroll
      for (int i = 0; i < VEC; ++i) o[i] = v[it][i] * rstd * wv[i];
      if (e[it] < dim) tm_store<VEC>(orow + e[it], o);
    }
  }
}

extern "C" int fg_stream_terms(const StreamTermsArgs* args, int n_rows, int act_dtype, int w_dtype, hipStream_t stream) {
  if (n_rows <= 0) return FG_OK;
  const StreamTermsArgs& a = *args;
  if (!a.h || a.dim <= 0 || a.dim > TM_MAX_DIM || a.n_terms < 0 || a.n_terms > TM_TERMS || (a.out[1] && !a.out[0]) ||
      (a.rows && !a.out[0]))
    return FG_ERR_ARG;
  for (int k = 0; k < 2; ++k)
    if (a.out[k] && !a.w[k]) return FG_ERR_ARG;
  for (int j = 0; j < a.n_terms; ++j)
    if ((!a.term[j].rows && !a.term[j].parts) || (!a.term[j].rows && a.term[j].n_parts < 1)) return FG_ERR_ARG;
#define GO(TA, TW, VEC, NIT) stream_terms_kernel<TA, TW, VEC, NIT><<<n_rows, TM_THREADS, 0, stream>>>(a)
#define LAUNCH(TA, TW)                                       \
  do {                                                       \
    if (a.dim % 8 == 0) {                                    \
      if (a.dim <= 8 * TM_THREADS) GO(TA, TW, 8, 1);         \
      else if (a.dim <= 16 * TM_THREADS) GO(TA, TW, 8, 2);   \
      else if (a.dim <= 32 * TM_THREADS) GO(TA, TW, 8, 4);   \
      else GO(TA, TW, 8, 8);                                 \
    } else if (a.dim <= 4 * TM_THREADS) {                    \
      GO(TA, TW, 1, 4);                                      \
    } else if (a.dim <= 16 * TM_THREADS) {                   \
      GO(TA, TW, 1, 16);                                     \
    } else {                                                 \
      GO(TA, TW, 1, 64);                                     \
    }                                                        \
  } while (0)
  if (act_dtype == FG_F32 && w_dtype == FG_F32) LAUNCH(float, float);
  else if (act_dtype == FG_BF16 && w_dtype == FG_BF16) LAUNCH(bf16_t, bf16_t);
  else if (act_dtype == FG_BF16 && w_dtype == FG_F32) LAUNCH(bf16_t, float);
  else if (act_dtype == FG_F32 && w_dtype == FG_BF16) LAUNCH(float, bf16_t);
  else return FG_ERR_ARG;
#undef LAUNCH
#undef GO
  return fg_launch_status();
}
