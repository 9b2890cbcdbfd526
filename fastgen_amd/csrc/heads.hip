// Per-head work around an attention or a recurrence that is no plain matrix product:
//
//  heads_prepare   what lies between the product that makes queries, keys and values and the
//                  attention: a causal convolution per channel, a bias, an RMS norm per head (over the
//                  head's first dimensions) or over all of a token's query (key) columns, the rotation of a run of dimensions, the queries to a buffer of their own (heads
//                  padded with zeros to the cache's head size) and keys and values into their cache
//                  pages.  A value is either columns of its own or the first dimensions of its
//                  processed key (a latent that serves as key and as value).
//  head_linear     y[t, h, :] = W_h x[t, h, :] with a matrix per head, an optional sigmoid gate per
//                  (token, head), and a run of x's columns behind the product's copied through.
//  head_norm_gate  RMS norm per head of fp32 rows times silu(gate) or sigmoid(gate); row_norm_gate: one norm over all
//                  of a row's heads.
//  head_diff_norm  the difference of two attention maps' outputs per head, divided by its root mean square.
//
// All arithmetic between a load and a store is fp32; a result is rounded once, at the store.
#include "common.h"
#include "kv_layout.h"
#include "conv_inputs.h"

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

#define HP_WAVES 4
#define HP_MAX_PAIRS 8  // pairs a lane holds: heads of up to 1,024 elements

struct PrepareArgs {
  const void* src; int src_stride;   // rows [T, src_stride]
  const float* bias;                 // per source column, or null
  int n_q, q_col, q_w, q_norm_dims; const float* q_norm_w;
  void* q_out; int q_out_stride, q_out_hw;  // queries: [T, q_out_stride], head h at h * q_out_hw, zeros behind q_w
  int n_kv, k_col, k_w, k_norm_dims; const float* k_norm_w;
  int v_col, v_w;                    // v_col < 0: a value is the first v_w elements of its processed key
  const float* table;                // [T, rotary_dim / 2, 2] cos, sin; null: nothing is rotated
  int rot_start, rotary_dim;         // pairs (rot_start + 2i, rot_start + 2i + 1) turn
  int rot_q, rot_k;                  // whether the query heads turn, and the key heads
  float eps;
  const int* slots; void* k_pages; void* v_pages; int page_size, hd_c;  // hd_c: the cache's head size
  int norm_plain;                    // a head with norm dims and no norm weight is divided by its root mean square
  const int* positions; float q_temp_coef; int q_temp_every;  // queries times 1 + coef * ln(floor((p + 1) / every) + 1)
  const void* v_first; int v_first_stride; float v_blend;     // values become (1 - v_blend) v + v_blend v_first[t, head, :]
  int row_norm;                      // the norms run over all n_q * q_w (n_kv * k_w) columns at once; weights [n * w]
  ConvIn conv;  // before anything else, on the query and key columns (channel = source column)
};

// A wave's (token, head): lane l holds the pairs l, l + 64, ..  CONV: the convolution comes first.  ROWN: the
// norm's factor comes from the caller (row_rstd_q, row_rstd_k).  NP: pairs a lane holds, for heads of up to 128 NP.
template <class TS, class TA, int NP, bool CONV, bool ROWN>
__device__ __forceinline__ void prepare_head(const PrepareArgs& a, int t, int job, float row_rstd_q, float row_rstd_k) {
  const int lane = threadIdx.x % FG_WAVE;
  const bool is_q = job < a.n_q;
  const int head = is_q ? job : job - a.n_q;
  int slot = -1;
  if (!is_q) {
    slot = a.slots[t];
    if (slot < 0) return;  // a token that writes nothing
  }
  const int w = is_q ? a.q_w : a.k_w;
  const int col = is_q ? a.q_col + head * a.q_w : a.k_col + head * a.k_w;
  const int norm_dims = is_q ? a.q_norm_dims : a.k_norm_dims;
  const float* norm_w = is_q ? a.q_norm_w : a.k_norm_w;
  const TS* row = (const TS*)a.src + (size_t)t * a.src_stride;
  float x[NP][2];
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < NP; ++j) {
    const int d = 2 * (lane + FG_WAVE * j);
    x[j][0] = x[j][1] = 0.f;
    if (d < w) {
      if (CONV) {
        conv_pair<TS>(a.conv, (const TS*)a.src, a.src_stride, t, col + d, x[j]);
      } else {
        x[j][0] = to_f<TS>(row[col + d]);
        x[j][1] = to_f<TS>(row[col + d + 1]);
      }
      if (a.bias) {
        x[j][0] += a.bias[col + d];
        x[j][1] += a.bias[col + d + 1];
      }
      if (d < norm_dims) ss += x[j][0] * x[j][0] + x[j][1] * x[j][1];
    }
  }
  // a query's temperature grows with the logarithm of its position, in steps of `every` positions
  const bool tempered = is_q && a.positions && a.q_temp_every > 0;  // uniform
  const float temp = tempered ? 1.f + a.q_temp_coef * logf((float)((a.positions[t] + 1) / a.q_temp_every) + 1.f) : 1.f;
  if (ROWN) {
    const float rstd = is_q ? row_rstd_q : row_rstd_k;
#pragma unroll
    for (int j = 0; j < NP; ++j) {
      const int d = 2 * (lane + FG_WAVE * j);
      if (d < w) {
        x[j][0] = x[j][0] * rstd * norm_w[head * w + d];
        x[j][1] = x[j][1] * rstd * norm_w[head * w + d + 1];
      }
    }
  } else if (norm_w || (a.norm_plain && norm_dims > 0)) {  // uniform
    ss = wave_sum(ss);
    const float rstd = rsqrtf(ss / (float)norm_dims + a.eps);
#pragma unroll
    for (int j = 0; j < NP; ++j) {
      const int d = 2 * (lane + FG_WAVE * j);
      if (d < norm_dims) {
        x[j][0] = x[j][0] * rstd * (norm_w ? norm_w[d] : 1.f);
        x[j][1] = x[j][1] * rstd * (norm_w ? norm_w[d + 1] : 1.f);
      }
    }
  }
  if (tempered) {
#pragma unroll
    for (int j = 0; j < NP; ++j) {
      x[j][0] *= temp;
      x[j][1] *= temp;
    }
  }
  if (a.table && (is_q ? a.rot_q : a.rot_k)) {  // uniform
#pragma unroll
    for (int j = 0; j < NP; ++j) {
      const int d = 2 * (lane + FG_WAVE * j);
      if (d >= a.rot_start && d < a.rot_start + a.rotary_dim && d < w) {
        const float2 cs = *(const float2*)(a.table + ((size_t)t * (a.rotary_dim / 2) + (d - a.rot_start) / 2) * 2);
        const float u = x[j][0], v = x[j][1];
        x[j][0] = u * cs.x - v * cs.y;
        x[j][1] = v * cs.x + u * cs.y;
      }
    }
  }
  if (is_q) {
    TA* o = (TA*)a.q_out + (size_t)t * a.q_out_stride + (size_t)head * a.q_out_hw;
#pragma unroll
    for (int j = 0; j < NP; ++j) {
      const int d = 2 * (lane + FG_WAVE * j);
      if (d < a.q_out_hw) {  // (x is zero from w on)
        o[d] = from_f<TA>(x[j][0]);
        o[d + 1] = from_f<TA>(x[j][1]);
      }
    }
    return;
  }
  const int page = slot / a.page_size, off = slot % a.page_size;
  const KvLayout lay(a.page_size, a.hd_c);
  const size_t head_elems = (size_t)a.page_size * a.hd_c;
  TA* kp = (TA*)a.k_pages + ((size_t)page * a.n_kv + head) * head_elems;
  TA* vp = (TA*)a.v_pages + ((size_t)page * a.n_kv + head) * head_elems;
#pragma unroll
  for (int j = 0; j < NP; ++j) {
    const int d = 2 * (lane + FG_WAVE * j);
    if (d < a.hd_c) {
      TA* dst = kp + lay.k_off(off, d);  // d is even: d + 1 lies in the same chunk of 8
      dst[0] = from_f<TA>(x[j][0]);
      dst[1] = from_f<TA>(x[j][1]);
      float v0 = 0.f, v1 = 0.f;
      if (d < a.v_w) {
        if (a.v_col < 0) {
          v0 = x[j][0];
          v1 = x[j][1];
        } else {
          const int c = a.v_col + head * a.v_w + d;
          v0 = to_f<TS>(row[c]) + (a.bias ? a.bias[c] : 0.f);
          v1 = to_f<TS>(row[c + 1]) + (a.bias ? a.bias[c + 1] : 0.f);
          if (a.v_first) {  // blended with the values that an earlier layer computed for this token
            const TS* f = (const TS*)a.v_first + (size_t)t * a.v_first_stride + head * a.v_w + d;
            v0 = (1.f - a.v_blend) * v0 + a.v_blend * to_f<TS>(f[0]);
            v1 = (1.f - a.v_blend) * v1 + a.v_blend * to_f<TS>(f[1]);
          }
        }
      }
      vp[lay.v_off(off, d)] = from_f<TA>(v0);
      vp[lay.v_off(off, d + 1)] = from_f<TA>(v1);
    }
  }
}

// grid (T, ceil((n_q + n_kv) / HP_WAVES)); a wave a (token, head)
template <class TS, class TA, int NP, bool CONV>
__global__ __launch_bounds__(HP_WAVES* FG_WAVE) void heads_prepare_kernel(const PrepareArgs a) {
  const int job = blockIdx.y * HP_WAVES + threadIdx.x / FG_WAVE;
  if (job >= a.n_q + a.n_kv) return;  // whole waves; no block barrier below
  prepare_head<TS, TA, NP, CONV, false>(a, blockIdx.x, job, 0.f, 0.f);
}

// Norms over all of a token's query columns and all its key columns: a workgroup a token, whose waves take the
// heads in turns once the two sums of squares are there.
#define HP_ROW_WAVES 8
template <class TS, class TA, int NP>
__global__ __launch_bounds__(HP_ROW_WAVES* FG_WAVE) void heads_prepare_row_kernel(const PrepareArgs a) {
  __shared__ float red[2][HP_ROW_WAVES];
  const int t = blockIdx.x, wave = threadIdx.x / FG_WAVE, lane = threadIdx.x % FG_WAVE;
  const TS* row = (const TS*)a.src + (size_t)t * a.src_stride;
  const int nq = a.n_q * a.q_w, nk = a.n_kv * a.k_w;
  float sq = 0.f, sk = 0.f;
  for (int i = threadIdx.x; i < nq; i += HP_ROW_WAVES * FG_WAVE) {
    const float v = to_f<TS>(row[a.q_col + i]) + (a.bias ? a.bias[a.q_col + i] : 0.f);
    sq += v * v;
  }
  for (int i = threadIdx.x; i < nk; i += HP_ROW_WAVES * FG_WAVE) {
    const float v = to_f<TS>(row[a.k_col + i]) + (a.bias ? a.bias[a.k_col + i] : 0.f);
    sk += v * v;
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if (lane == 0) {
    red[0][wave] = sq;
    red[1][wave] = sk;
  }
  __syncthreads();
  sq = sk = 0.f;
#pragma unroll
  for (int i = 0; i < HP_ROW_WAVES; ++i) {
    sq += red[0][i];
    sk += red[1][i];
  }
  const float rq = nq ? rsqrtf(sq / (float)nq + a.eps) : 0.f, rk = nk ? rsqrtf(sk / (float)nk + a.eps) : 0.f;
  for (int job = wave; job < a.n_q + a.n_kv; job += HP_ROW_WAVES) prepare_head<TS, TA, NP, false, true>(a, t, job, rq, rk);
}

extern "C" int fg_heads_prepare(const PrepareArgs* args, int n_tokens, int src_dtype, int act_dtype,
                                hipStream_t stream) {
  if (n_tokens <= 0) return FG_OK;
  const PrepareArgs& a = *args;
  const int lim = 2 * FG_WAVE * HP_MAX_PAIRS;
  if (a.n_q < 0 || a.n_kv < 0 || a.n_q + a.n_kv <= 0 || !a.src) return FG_ERR_ARG;
  if (a.n_q && (a.q_w <= 0 || a.q_w % 2 || a.q_w > lim || a.q_out_hw < a.q_w || a.q_out_hw % 2 || a.q_out_hw > lim ||
                !a.q_out || a.q_norm_dims > a.q_w || a.q_norm_dims % 2))
    return FG_ERR_ARG;
  if (a.n_kv && (a.k_w <= 0 || a.k_w % 2 || a.hd_c < a.k_w || a.hd_c % 8 || a.hd_c > lim || a.v_w <= 0 || a.v_w % 2 ||
                 a.v_w > a.hd_c || (a.v_col < 0 && a.v_w > a.k_w) || a.page_size <= 0 || a.page_size % 8 ||
                 !a.slots || !a.k_pages || !a.v_pages || a.k_norm_dims > a.k_w || a.k_norm_dims % 2))
    return FG_ERR_ARG;
  if (a.table && (a.rot_start < 0 || a.rot_start % 2 || a.rotary_dim <= 0 || a.rotary_dim % 2)) return FG_ERR_ARG;
  const int jobs = a.n_q + a.n_kv;
  dim3 grid(n_tokens, (jobs + HP_WAVES - 1) / HP_WAVES);
  if (grid.y > 65535) return FG_ERR_ARG;
  if (a.conv.w && (!fg_conv_ok(a.conv) || (a.n_q && a.q_col + a.n_q * a.q_w > a.conv.channels) ||
                   (a.n_kv && a.k_col + a.n_kv * a.k_w > a.conv.channels)))
    return FG_ERR_ARG;
  if (a.row_norm && (a.conv.w || (a.n_q && !a.q_norm_w) || (a.n_kv && !a.k_norm_w))) return FG_ERR_ARG;
  int widest = a.n_q ? (a.q_w > a.q_out_hw ? a.q_w : a.q_out_hw) : 0;
  if (a.n_kv && a.hd_c > widest) widest = a.hd_c;
#define GO1(TS, TA, NP)                                                                                           \
  do {                                                                                                            \
    if (a.row_norm) heads_prepare_row_kernel<TS, TA, NP><<<n_tokens, HP_ROW_WAVES * FG_WAVE, 0, stream>>>(a);     \
    else if (a.conv.w) heads_prepare_kernel<TS, TA, NP, true><<<grid, HP_WAVES * FG_WAVE, 0, stream>>>(a);        \
    else heads_prepare_kernel<TS, TA, NP, false><<<grid, HP_WAVES * FG_WAVE, 0, stream>>>(a);                     \
  } while (0)
#define GO(TS, TA)                                                  \
  do {                                                              \
    if (widest <= 2 * FG_WAVE) GO1(TS, TA, 1);                      \
    else if (widest <= 4 * FG_WAVE) GO1(TS, TA, 2);                 \
    else GO1(TS, TA, HP_MAX_PAIRS);                                 \
  } while (0)
  if (src_dtype == FG_F32 && act_dtype == FG_F32) GO(float, float);
  else if (src_dtype == FG_F32 && act_dtype == FG_BF16) GO(float, bf16_t);
  else if (src_dtype == FG_BF16 && act_dtype == FG_BF16) GO(bf16_t, bf16_t);
  else return FG_ERR_ARG;
#undef GO
#undef GO1
  return fg_launch_status();
}

// ------------------------------------------------------------------ head_linear
struct HeadLinearArgs {
  const void* x; int x_stride, x_hs;   // x[t, h, k] at t * x_stride + h * x_hs + k
  const void* w;                       // [H, N, K]
  void* y; int y_stride, y_hs;         // y[t, h, n] at t * y_stride + h * y_hs + n
  const float* gate; int gate_stride;  // gate[t * gate_stride + h] or null: y *= sigmoid(gate)
  int T, H, N, K;
  int tail, y_hw;  // y[t, h, N + j] = x[t, h, K + j] for j < tail; zeros from N + tail to y_hw
  const float* bias;  // [H, N] or null, added to the product
};

// Any dtype: grid (T, H), 256 threads; x's head goes through LDS, a thread an output element.
#define HL_MAX_K 1024
template <class T, class TY>
__global__ __launch_bounds__(256) void head_linear_kernel(const HeadLinearArgs a) {
  __shared__ float x_s[HL_MAX_K];
  const int t = blockIdx.x, h = blockIdx.y;
  const T* x = (const T*)a.x + (size_t)t * a.x_stride + (size_t)h * a.x_hs;
  for (int k = threadIdx.x; k < a.K; k += 256) x_s[k] = to_f<T>(x[k]);
  __syncthreads();
  float gv = 1.f;
  if (a.gate) gv = 1.f / (1.f + expf(-a.gate[(size_t)t * a.gate_stride + h]));
  TY* y = (TY*)a.y + (size_t)t * a.y_stride + (size_t)h * a.y_hs;
  const T* w = (const T*)a.w + (size_t)h * a.N * a.K;
  for (int n = threadIdx.x; n < a.y_hw; n += 256) {
    float acc = 0.f;
    if (n < a.N) {
      const T* wr = w + (size_t)n * a.K;
      for (int k = 0; k < a.K; ++k) acc += to_f<T>(wr[k]) * x_s[k];  // k ascending
      if (a.bias) acc += a.bias[(size_t)h * a.N + n];
      acc *= gv;
    } else if (n < a.N + a.tail) {
      acc = to_f<T>(x[a.K + n - a.N]);
    }
    y[n] = from_f<TY>(acc);
  }
}

// bfloat16 on the matrix cores: grid (ceil(T / 64), ceil(N / 64), H), 4 waves; a wave takes 16
// output channels and 64 tokens (four blocks of 16), operands straight from memory.  K % 8 == 0 and
// rows of x 16-byte aligned.  acc[mb][i] = y[token 16 mb + (lane & 15)][channel 4 (lane >> 4) + i].
template <class TY>
__global__ __launch_bounds__(256) void head_linear_mfma_kernel(const HeadLinearArgs a) {
  const int lane = threadIdx.x % FG_WAVE, wave = threadIdx.x / FG_WAVE;
  const int r16 = lane & 15, g = lane >> 4;
  const int m0 = blockIdx.x * 64, n0 = (blockIdx.y * 4 + wave) * 16, h = blockIdx.z;
  const bf16_t* xh = (const bf16_t*)a.x + (size_t)h * a.x_hs;
  if (n0 < a.N) {  // whole waves
    const bf16_t* wrow = (const bf16_t*)a.w + ((size_t)h * a.N + min(n0 + r16, a.N - 1)) * a.K;
    const bf16_t* xrow[4];
#pragma unroll
    for (int mb = 0; mb < 4; ++mb) xrow[mb] = xh + (size_t)min(m0 + 16 * mb + r16, a.T - 1) * a.x_stride;
    f32x4 acc[4];
#pragma unroll
    for (int mb = 0; mb < 4; ++mb) acc[mb] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < a.K; k0 += 32) {
      const int kk = k0 + 8 * g;
      bf16x8 wa, xb[4];
      if (kk < a.K) {
        wa = *(const bf16x8*)(wrow + kk);
#pragma unroll
        for (int mb = 0; mb < 4; ++mb) xb[mb] = *(const bf16x8*)(xrow[mb] + kk);
      } else {
#pragma unroll
        for (int i = 0; i < 8; ++i) wa[i] = (__bf16)0.f;
#pragma unroll
        for (int mb = 0; mb < 4; ++mb) xb[mb] = wa;
      }
#pragma unroll
      for (int mb = 0; mb < 4; ++mb) acc[mb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wa, xb[mb], acc[mb], 0, 0, 0);
    }
#pragma unroll
    for (int mb = 0; mb < 4; ++mb) {
      const int t = m0 + 16 * mb + r16;
      if (t >= a.T) continue;
      float gv = 1.f;
      if (a.gate) gv = 1.f / (1.f + __expf(-a.gate[(size_t)t * a.gate_stride + h]));
      TY* y = (TY*)a.y + (size_t)t * a.y_stride + (size_t)h * a.y_hs;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int n = n0 + 4 * g + i;
        if (n < a.N) y[n] = from_f<TY>((acc[mb][i] + (a.bias ? a.bias[(size_t)h * a.N + n] : 0.f)) * gv);
      }
    }
  }
  if (blockIdx.y == 0) {  // what lies behind the product: copied columns, then zeros
    const int extra = a.y_hw - a.N;
    for (int e = threadIdx.x; e < 64 * extra; e += 256) {
      const int t = m0 + e / extra, j = e % extra;
      if (t >= a.T) break;
      const bf16_t v = j < a.tail ? xh[(size_t)t * a.x_stride + a.K + j] : (bf16_t)0.f;
      ((TY*)a.y)[(size_t)t * a.y_stride + (size_t)h * a.y_hs + a.N + j] = from_f<TY>(to_f<bf16_t>(v));
    }
  }
}

// dtype: of x and w; out_dtype: of y, the same or fp32
extern "C" int fg_head_linear(const HeadLinearArgs* args, int dtype, int out_dtype, int use_mfma, hipStream_t stream) {
  const HeadLinearArgs& a = *args;
  if (a.T <= 0) return FG_OK;
  if (a.H <= 0 || a.N <= 0 || a.K <= 0 || a.tail < 0 || a.y_hw < a.N + a.tail || a.x_hs < a.K + a.tail ||
      a.y_hs < a.y_hw || !a.x || !a.w || !a.y)
    return FG_ERR_ARG;
  if (use_mfma) {
    if (dtype != FG_BF16 || a.K % 8 || a.x_stride % 8 || a.x_hs % 8 || a.H > 65535 || (a.N + 63) / 64 > 65535)
      return FG_ERR_ARG;
    const dim3 grid((a.T + 63) / 64, (a.N + 63) / 64, a.H);
    if (out_dtype == FG_BF16) head_linear_mfma_kernel<bf16_t><<<grid, 256, 0, stream>>>(a);
    else if (out_dtype == FG_F32) head_linear_mfma_kernel<float><<<grid, 256, 0, stream>>>(a);
    else return FG_ERR_ARG;
    return fg_launch_status();
  }
  if (a.K > HL_MAX_K || a.H > 65535) return FG_ERR_ARG;
  const dim3 grid(a.T, a.H);
  if (dtype == FG_F32 && out_dtype == FG_F32) head_linear_kernel<float, float><<<grid, 256, 0, stream>>>(a);
  else if (dtype == FG_BF16 && out_dtype == FG_BF16) head_linear_kernel<bf16_t, bf16_t><<<grid, 256, 0, stream>>>(a);
  else if (dtype == FG_BF16 && out_dtype == FG_F32) head_linear_kernel<bf16_t, float><<<grid, 256, 0, stream>>>(a);
  else return FG_ERR_ARG;
  return fg_launch_status();
}

// ---------------------------------------------------------------- head_norm_gate
// out[t, h, :] = x[t, h, :] * rsqrt(mean(x[t, h, :]^2) + eps) * w * silu(g[t, h, :]) * out_scale; x fp32 [T, H * e],
// g (act dtype) columns of a wider row.  `sigmoid`: the gate's sigmoid in its silu's place.  grid (T, ceil(H / 4)); a wave a (token, head).
#define HN_MAX 16  // elements a lane holds: heads of up to 1,024
template <class TA, class TG>
__global__ __launch_bounds__(HP_WAVES* FG_WAVE) void head_norm_gate_kernel(
    const float* __restrict__ x, const float* __restrict__ w, const TG* __restrict__ gate, int gate_stride,
    TA* __restrict__ out, int out_stride, int H, int e, float eps, float out_scale, int sigmoid) {
  const int lane = threadIdx.x % FG_WAVE, wave = threadIdx.x / FG_WAVE;
  const int t = blockIdx.x, h = blockIdx.y * HP_WAVES + wave;
  if (h >= H) return;
  const float* xr = x + ((size_t)t * H + h) * e;
  float v[HN_MAX];
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < HN_MAX; ++j) {
    const int d = lane + FG_WAVE * j;
    v[j] = d < e ? xr[d] : 0.f;
    ss += v[j] * v[j];
  }
  ss = wave_sum(ss);
  const float rstd = rsqrtf(ss / (float)e + eps) * out_scale;
  const TG* gr = gate + (size_t)t * gate_stride + (size_t)h * e;
  TA* o = out + (size_t)t * out_stride + (size_t)h * e;
#pragma unroll
  for (int j = 0; j < HN_MAX; ++j) {
    const int d = lane + FG_WAVE * j;
    if (d < e) {
      const float gv = to_f<TG>(gr[d]);
      o[d] = from_f<TA>(v[j] * rstd * w[d] * ((sigmoid ? 1.f : gv) / (1.f + expf(-gv))));
    }
  }
}

extern "C" int fg_head_norm_gate(const float* x, const float* w, const void* gate, int gate_stride, void* out,
                                 int out_stride, int n_tokens, int H, int e, float eps, float out_scale, int sigmoid, int act_dtype,
                                 int gate_dtype, hipStream_t stream) {
  if (n_tokens <= 0) return FG_OK;
  if (H <= 0 || e <= 0 || e > HN_MAX * FG_WAVE || gate_stride < H * e || out_stride < H * e || (H + HP_WAVES - 1) / HP_WAVES > 65535)
    return FG_ERR_ARG;
  dim3 grid(n_tokens, (H + HP_WAVES - 1) / HP_WAVES);
#define GO(TA, TG)                                                                                             \
  head_norm_gate_kernel<TA, TG><<<grid, HP_WAVES * FG_WAVE, 0, stream>>>(x, w, (const TG*)gate, gate_stride,   \
                                                                         (TA*)out, out_stride, H, e, eps, out_scale, sigmoid)
  if (act_dtype == FG_F32 && gate_dtype == FG_F32) GO(float, float);
  else if (act_dtype == FG_BF16 && gate_dtype == FG_BF16) GO(bf16_t, bf16_t);
  else if (act_dtype == FG_BF16 && gate_dtype == FG_F32) GO(bf16_t, float);
  else return FG_ERR_ARG;
#undef GO
  return fg_launch_status();
}

// ---------------------------------------------------------------- row_norm_gate
// out[t, :] = x[t, :] * rsqrt(mean(x[t, :]^2) + eps) * w * sigmoid(g[t, :]) * out_scale over W columns; x fp32 [T, W], g
// (fp32) columns of a wider row.  A workgroup a row, which it keeps in registers: NIT elements a thread.
#define RN_THREADS 256
#define RN_MAX 64
template <class TA, int NIT>
__global__ __launch_bounds__(RN_THREADS) void row_norm_gate_kernel(
    const float* __restrict__ x, const float* __restrict__ w, const float* __restrict__ gate, int gate_stride,
    TA* __restrict__ out, int out_stride, int W, float eps, float out_scale) {
  __shared__ float red[16];
  const size_t t = blockIdx.x;
  const float* xr = x + t * W;
  const float* gr = gate + t * gate_stride;
  float v[NIT], gv[NIT], wv[NIT], ss = 0.f;
#pragma unroll
  for (int j = 0; j < NIT; ++j) {  // (never conditional: beyond the row its last element, which counts for nothing)
    const int c = min((int)threadIdx.x + RN_THREADS * j, W - 1);
    v[j] = xr[c];
    gv[j] = gr[c];
    wv[j] = w[c];
  }
#pragma unroll
  for (int j = 0; j < NIT; ++j)
    if ((int)threadIdx.x + RN_THREADS * j < W) ss += v[j] * v[j];
  ss = block_sum(ss, red);
  const float rstd = rsqrtf(ss / (float)W + eps) * out_scale;
#pragma unroll
  for (int j = 0; j < NIT; ++j) {
    const int c = threadIdx.x + RN_THREADS * j;
    if (c < W) out[t * out_stride + c] = from_f<TA>(v[j] * rstd * wv[j] / (1.f + expf(-gv[j])));
  }
}

extern "C" int fg_row_norm_gate(const float* x, const float* w, const float* gate, int gate_stride, void* out, int out_stride,
                                int n_tokens, int W, float eps, float out_scale, int act_dtype, hipStream_t stream) {
  if (n_tokens <= 0) return FG_OK;
  if (W <= 0 || W > RN_MAX * RN_THREADS || gate_stride < W || out_stride < W) return FG_ERR_ARG;
#define GO(TA, NIT) row_norm_gate_kernel<TA, NIT><<<n_tokens, RN_THREADS, 0, stream>>>(x, w, gate, gate_stride, (TA*)out, out_stride, W, eps, out_scale)
#define LAUNCH(TA)                                  \
  do {                                              \
    if (W <= 2 * RN_THREADS) GO(TA, 2);             \
    else if (W <= 8 * RN_THREADS) GO(TA, 8);        \
    else if (W <= 16 * RN_THREADS) GO(TA, 16);      \
    else GO(TA, RN_MAX);                            \
  } while (0)
  if (act_dtype == FG_F32) LAUNCH(float);
  else if (act_dtype == FG_BF16) LAUNCH(bf16_t);
  else return FG_ERR_ARG;
#undef LAUNCH
#undef GO
  return fg_launch_status();
}

// ---------------------------------------------------------------- head_diff_norm
// Two attention maps a head, one value: out[t, h, :] = n(a1 - lam * a2) * out_scale with
// n(o) = o * rsqrt(mean(o^2) + eps) over the head's e values (no weight).  `att` holds 2 H heads of `hw`
// columns (the first e are the head's output): the heads of a key/value group of `group` query heads lie
// as [map 1 of the group's heads | map 2 of the group's heads], so a1 of head h is head
// (h / group) * 2 * group + h % group of `att` and a2 lies `group` heads behind it.  All in fp32, one
// rounding at the store.  grid (T, ceil(H / 4)); a wave a (token, head).
template <class TA>
__global__ __launch_bounds__(HP_WAVES* FG_WAVE) void head_diff_norm_kernel(
    const TA* __restrict__ att, int att_stride, int hw, TA* __restrict__ out, int out_stride, int H, int group, int e,
    float lam, float eps, float out_scale) {
  const int lane = threadIdx.x % FG_WAVE, wave = threadIdx.x / FG_WAVE;
  const int t = blockIdx.x, h = blockIdx.y * HP_WAVES + wave;
  if (h >= H) return;
  const TA* a1 = att + (size_t)t * att_stride + (size_t)((h / group) * 2 * group + h % group) * hw;
  const TA* a2 = a1 + (size_t)group * hw;
  float v[HN_MAX];
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < HN_MAX; ++j) {
    const int d = lane + FG_WAVE * j;
    v[j] = d < e ? to_f<TA>(a1[d]) - lam * to_f<TA>(a2[d]) : 0.f;
    ss += v[j] * v[j];
  }
  ss = wave_sum(ss);
  const float mul = rsqrtf(ss / (float)e + eps) * out_scale;
  TA* o = out + (size_t)t * out_stride + (size_t)h * e;
#pragma unroll
  for (int j = 0; j < HN_MAX; ++j) {
    const int d = lane + FG_WAVE * j;
    if (d < e) o[d] = from_f<TA>(v[j] * mul);
  }
}

extern "C" int fg_head_diff_norm(const void* att, int att_stride, int hw, void* out, int out_stride, int n_tokens, int H,
                                 int group, int e, float lam, float eps, float out_scale, int act_dtype,
                                 hipStream_t stream) {
  if (n_tokens <= 0) return FG_OK;
  if (H <= 0 || group <= 0 || H % group || e <= 0 || e > HN_MAX * FG_WAVE || hw < e || att_stride < 2 * H * hw ||
      out_stride < H * e || (H + HP_WAVES - 1) / HP_WAVES > 65535)
    return FG_ERR_ARG;
  dim3 grid(n_tokens, (H + HP_WAVES - 1) / HP_WAVES);
  if (act_dtype == FG_F32)
    head_diff_norm_kernel<float><<<grid, HP_WAVES * FG_WAVE, 0, stream>>>((const float*)att, att_stride, hw, (float*)out,
                                                                         out_stride, H, group, e, lam, eps, out_scale);
  else if (act_dtype == FG_BF16)
    head_diff_norm_kernel<bf16_t><<<grid, HP_WAVES * FG_WAVE, 0, stream>>>((const bf16_t*)att, att_stride, hw, (bf16_t*)out,
                                                                          out_stride, H, group, e, lam, eps, out_scale);
  else
    return FG_ERR_ARG;
  return fg_launch_status();
}
