// The gated delta rule: a state S [d, e] per head in fp32, kept per request and carried from step to step.
//
//   S <- g_t S;   u_t = beta_t (v_t - S^T k_t);   S <- S + k_t u_t^T;   o_t = S^T q_t
//
// g_t is a number per head, or a number per head and key channel: row c of S then fades by its own g_t[c].
//
//  delta_prepare  what the recurrence takes of a token, from the rows of the product: a causal convolution per
//                 channel and SiLU on q, k and v; q and k as unit vectors per head (q times q_scale); the write
//                 strength beta = sigmoid(b) and the decay's logarithm log g = -exp(A_log) softplus(a + dt_bias) per
//                 head.  One fp32 row a token: [q | k | v | beta | log g].  A wave a (token, head).  Decays per channel
//                 are the caller's: their logarithms stand anywhere in the row, n_v * d of them.
//  delta_scan     the recurrence token by token.  Column c of S needs k, q and v[c] only, so a wave owns eight value
//                 channels of a head: lane l holds column l & 7 and the key channels rg * rpl .. (rg = l >> 3) of it in
//                 registers.  S^T k is a sum over the lanes of a column on the chain; S^T q is not, its sums are
//                 exchanged for a whole run of tokens at once.  Operands of the next run fly while one is computed.
//                 Every sum runs in an order fixed by the sizes: the result does not depend on the batch or the cut.
//  delta_chunk_*  long prompts, 64 tokens at a time as matrix products (the WY form of the products of the tokens'
//                 rank-one changes), see below: the same within rounding.
#include "common.h"
#include "conv_inputs.h"

#define DP_WAVES 4
#define DP_MAX_PAIRS 8  // heads of up to 1,024 elements

struct DeltaPrepareArgs {
  const void* src; int src_stride;       // [T, q | k | v ...]: q from column 0, k and v right behind
  int n_qk, d, n_v, e;                   // query/key heads of d, value heads of e
  ConvIn conv;                           // over the q, k and v columns
  int b_col, a_col;                      // columns of the beta and decay logits (n_v each); a_col < 0: no decays here
  const float* decay_rate;               // [n_v]: exp(A_log)
  const float* dt_bias;                  // [n_v]
  float q_scale, unit_eps;
  float* out; int out_stride;            // [T, 2 n_qk d + n_v e + 2 n_v]
};

// grid (T, ceil((2 n_qk + n_v + 1) / 4)); the last job of a token is its scalars, a lane a head
template <class TS, int NP>
__global__ __launch_bounds__(DP_WAVES* FG_WAVE) void delta_prepare_kernel(const DeltaPrepareArgs a) {
  const int lane = threadIdx.x % FG_WAVE, t = blockIdx.x, job = blockIdx.y * DP_WAVES + threadIdx.x / FG_WAVE;
  const int qk_jobs = 2 * a.n_qk, v_base = qk_jobs * a.d;
  if (job > qk_jobs + a.n_v) return;  // whole waves; no block barrier below
  const TS* src = (const TS*)a.src;
  float* out = a.out + (size_t)t * a.out_stride;
  if (job == qk_jobs + a.n_v) {
    const TS* row = src + (size_t)t * a.src_stride;
    float* so = out + v_base + a.n_v * a.e;
    for (int h = lane; h < a.n_v; h += FG_WAVE) {
      const float b = to_f<TS>(row[a.b_col + h]);
      so[h] = 1.f / (1.f + expf(-b));
      if (a.a_col < 0) continue;
      const float x = to_f<TS>(row[a.a_col + h]) + a.dt_bias[h];
      so[a.n_v + h] = -a.decay_rate[h] * (fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))));
    }
    return;
  }
  const bool is_v = job >= qk_jobs;
  const int w = is_v ? a.e : a.d;
  const int col = is_v ? v_base + (job - qk_jobs) * a.e : job * a.d;
  float x[NP][2];
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < NP; ++j) {
    const int c = 2 * (lane + FG_WAVE * j);
    x[j][0] = x[j][1] = 0.f;
    if (c < w) {
      conv_pair<TS>(a.conv, src, a.src_stride, t, col + c, x[j]);
#pragma unroll
      for (int i = 0; i < 2; ++i) x[j][i] = x[j][i] / (1.f + expf(-x[j][i]));
      ss += x[j][0] * x[j][0] + x[j][1] * x[j][1];
    }
  }
  float mul = 1.f;
  if (!is_v) {  // uniform
    ss = wave_sum(ss);
    mul = rsqrtf(ss + a.unit_eps) * (job < a.n_qk ? a.q_scale : 1.f);
  }
#pragma unroll
  for (int j = 0; j < NP; ++j) {
    const int c = 2 * (lane + FG_WAVE * j);
    if (c < w) *(float2*)(out + col + c) = make_float2(x[j][0] * mul, x[j][1] * mul);
  }
}

extern "C" int fg_delta_prepare(const DeltaPrepareArgs* args, int n_tokens, int src_dtype, hipStream_t stream) {
  if (n_tokens <= 0) return FG_OK;
  const DeltaPrepareArgs& a = *args;
  const int lim = 2 * FG_WAVE * DP_MAX_PAIRS;
  if (a.n_qk <= 0 || a.n_v <= 0 || a.d <= 0 || a.d % 2 || a.d > lim || a.e <= 0 || a.e % 2 || a.e > lim || !a.src || !a.out ||
      (a.a_col >= 0 && (!a.decay_rate || !a.dt_bias)) || !a.conv.w || !fg_conv_ok(a.conv) || a.conv.channels < 2 * a.n_qk * a.d + a.n_v * a.e ||
      a.out_stride % 2 || a.out_stride < 2 * a.n_qk * a.d + a.n_v * (a.e + (a.a_col < 0 ? 1 : 2)))
    return FG_ERR_ARG;
  const dim3 grid(n_tokens, (2 * a.n_qk + a.n_v + 1 + DP_WAVES - 1) / DP_WAVES);
  if (grid.y > 65535) return FG_ERR_ARG;
  const int widest = a.d > a.e ? a.d : a.e;
#define GO(TS)                                                                                                 \
  do {                                                                                                         \
    if (widest <= 2 * FG_WAVE) delta_prepare_kernel<TS, 1><<<grid, DP_WAVES * FG_WAVE, 0, stream>>>(a);        \
    else if (widest <= 4 * FG_WAVE) delta_prepare_kernel<TS, 2><<<grid, DP_WAVES * FG_WAVE, 0, stream>>>(a);   \
    else delta_prepare_kernel<TS, DP_MAX_PAIRS><<<grid, DP_WAVES * FG_WAVE, 0, stream>>>(a);                   \
  } while (0)
  if (src_dtype == FG_F32) GO(float);
  else if (src_dtype == FG_BF16) GO(bf16_t);
  else return FG_ERR_ARG;
#undef GO
  return fg_launch_status();
}

// ------------------------------------------------------------------- scan
struct DeltaScanArgs {
  const float* rows; int stride;         // delta_prepare's rows
  int n_qk, d, n_v, e;
  float* state; long long slot_stride;   // S of slot s, head h at s * slot_stride + h * d * e, [d, e]
  const int* slot_ids; const int* q_start;
  float* out;                            // [T, n_v * e]
  int g_col, per_channel;                // where the decays' logarithms begin; n_v of them, or n_v * d
};

// The sum over the eight lanes that hold a column (lane % 8 equal), in every one of them: lanes 8 apart by a
// rotation within a row of 16, then rows and halves exchanged in the vector unit.
__device__ __forceinline__ float column_sum(float v) {
  v += __uint_as_float(__builtin_amdgcn_update_dpp(0, __float_as_uint(v), 0x128 /* row_ror:8 */, 0xf, 0xf, false));
  const auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  v = __uint_as_float(a[0]) + __uint_as_float(a[1]);
  const auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  return __uint_as_float(b[0]) + __uint_as_float(b[1]);
}

#define DS_TOKENS_FOR(RPL) ((RPL) <= 16 ? 8 : 4)  // tokens staged at a time

// grid (B, n_v, ceil(e / 8)), one wave.  RPL >= ceil(d / 8), a multiple of 4; NJ: staged elements a lane holds of k
// and of q (CH, decays per channel: and of g) per token.
template <int RPL, bool CH>
__global__ __launch_bounds__(FG_WAVE) void delta_scan_kernel(const DeltaScanArgs a) {
  constexpr int RUN = DS_TOKENS_FOR(RPL);
  constexpr int NJ = (RPL + 7) / 8;  // 64 lanes, up to 8 RPL channels
  // [RUN][NS][8 parts of RPL + 4]: k, q (and g); key channel r of part p = r / rpl at p * (RPL + 4) + r % rpl, zeros behind rpl
  constexpr int PS = RPL + 4, VS = 8 * PS, NS = CH ? 3 : 2;
  __shared__ __attribute__((aligned(16))) float lds[RUN * NS * VS];
  const int lane = threadIdx.x;
  const int b = blockIdx.x, h = blockIdx.y;
  const int rg = lane >> 3, col = blockIdx.z * 8 + (lane & 7);
  const bool col_ok = col < a.e;
  const int d = a.d, e = a.e, rpl = (d + 7) / 8, r0 = rg * rpl;
  const int hq = h / (a.n_v / a.n_qk);
  const int t_begin = a.q_start[b], t_end = a.q_start[b + 1];
  if (t_begin >= t_end) return;  // uniform
  float* S_mem = a.state + (size_t)a.slot_ids[b] * a.slot_stride + (size_t)h * d * e;
  float S[RPL];
#pragma unroll
  for (int i = 0; i < RPL; ++i) S[i] = (i < rpl && r0 + i < d && col_ok) ? S_mem[(size_t)(r0 + i) * e + col] : 0.f;
  for (int i = lane; i < RUN * NS * VS; i += FG_WAVE) lds[i] = 0.f;
  int src[NJ], dst[NJ];
  bool mine[NJ];
#pragma unroll
  for (int j = 0; j < NJ; ++j) {
    const int r = lane + FG_WAVE * j;
    mine[j] = r < d;
    src[j] = hq * d + min(r, d - 1);
    dst[j] = (r / rpl) * PS + r % rpl;
  }
  const int k_col = a.n_qk * d, v_col = 2 * k_col + h * e + min(col, e - 1);
  const int b_col = 2 * k_col + a.n_v * e + h, g_col = a.g_col + (CH ? h * d : h);
  float pk[RUN][NJ], pq[RUN][NJ], pv[RUN], pb[RUN], pg[RUN][CH ? NJ : 1];
  auto fetch = [&](int t0) {
#pragma unroll
    for (int tt = 0; tt < RUN; ++tt) {
      const float* row = a.rows + (size_t)min(t0 + tt, t_end - 1) * a.stride;
#pragma unroll
      for (int j = 0; j < NJ; ++j) {
        pk[tt][j] = row[k_col + src[j]];
        pq[tt][j] = row[src[j]];
        if (CH) pg[tt][j] = row[g_col + min(lane + FG_WAVE * j, d - 1)];  // (its logarithm)
      }
      pv[tt] = row[v_col];
      pb[tt] = row[b_col];
      if (!CH) pg[tt][0] = row[g_col];
    }
  };
  fetch(t_begin);
  for (int t0 = t_begin; t0 < t_end; t0 += RUN) {
    const int n = min(RUN, t_end - t0);
    __syncthreads();  // the run before has been read
    float v[RUN], beta[RUN], g[RUN];
#pragma unroll
    for (int tt = 0; tt < RUN; ++tt) {
      v[tt] = pv[tt];
      beta[tt] = pb[tt];
      if (!CH) g[tt] = expf(pg[tt][0]);
#pragma unroll
      for (int j = 0; j < NJ; ++j) {
        if (mine[j]) {
          lds[tt * NS * VS + dst[j]] = pk[tt][j];
          lds[tt * NS * VS + VS + dst[j]] = pq[tt][j];
          if (CH) lds[tt * NS * VS + 2 * VS + dst[j]] = expf(pg[tt][j]);
        }
      }
    }
    __syncthreads();
    if (t0 + RUN < t_end) fetch(t0 + RUN);
    float acc[RUN];
#pragma unroll
    for (int tt = 0; tt < RUN; ++tt) {
      acc[tt] = 0.f;
      if (tt < n) {  // uniform
        const float4* kp = (const float4*)(lds + tt * NS * VS + rg * PS);
        const float4* qp = (const float4*)(lds + tt * NS * VS + VS + rg * PS);
        const float4* gp = (const float4*)(lds + tt * NS * VS + (NS - 1) * VS + rg * PS);
        float kv[RPL], part[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i4 = 0; i4 < RPL / 4; ++i4) {
          const float4 k4 = kp[i4];
          kv[4 * i4] = k4.x; kv[4 * i4 + 1] = k4.y; kv[4 * i4 + 2] = k4.z; kv[4 * i4 + 3] = k4.w;
          const float4 g4 = CH ? gp[i4] : make_float4(g[tt], g[tt], g[tt], g[tt]);
          const float gg[4] = {g4.x, g4.y, g4.z, g4.w};
#pragma unroll
          for (int u = 0; u < 4; ++u) {
            S[4 * i4 + u] *= gg[u];
            part[u] += S[4 * i4 + u] * kv[4 * i4 + u];
          }
        }
        const float ks = column_sum((part[0] + part[1]) + (part[2] + part[3]));
        const float uv = beta[tt] * (v[tt] - ks);
        float op[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i4 = 0; i4 < RPL / 4; ++i4) {
          const float4 q4 = qp[i4];
          const float qq[4] = {q4.x, q4.y, q4.z, q4.w};
#pragma unroll
          for (int u = 0; u < 4; ++u) {
            S[4 * i4 + u] += kv[4 * i4 + u] * uv;
            op[u] += S[4 * i4 + u] * qq[u];
          }
        }
        acc[tt] = (op[0] + op[1]) + (op[2] + op[3]);
      }
    }
#pragma unroll
    for (int tt = 0; tt < RUN; ++tt) acc[tt] = column_sum(acc[tt]);
    if (rg == 0 && col_ok) {
#pragma unroll
      for (int tt = 0; tt < RUN; ++tt)
        if (tt < n) a.out[(size_t)(t0 + tt) * ((size_t)a.n_v * e) + h * e + col] = acc[tt];
    }
  }
#pragma unroll
  for (int i = 0; i < RPL; ++i)
    if (i < rpl && r0 + i < d && col_ok) S_mem[(size_t)(r0 + i) * e + col] = S[i];
}

static bool delta_scan_ok(const DeltaScanArgs& a, int n_seqs) {
  return a.n_qk > 0 && a.n_v > 0 && a.n_v % a.n_qk == 0 && a.d > 0 && a.d <= 512 && a.e > 0 && a.n_v <= 65535 &&
         n_seqs <= 65535 && (a.e + 7) / 8 <= 65535 && a.rows && a.state && a.slot_ids && a.q_start && a.out &&
         a.g_col >= 2 * a.n_qk * a.d + a.n_v * (a.e + 1) && a.stride >= a.g_col + a.n_v * (a.per_channel ? a.d : 1);
}

extern "C" int fg_delta_scan(const DeltaScanArgs* args, int n_seqs, hipStream_t stream) {
  if (n_seqs <= 0) return FG_OK;
  const DeltaScanArgs& a = *args;
  if (!delta_scan_ok(a, n_seqs)) return FG_ERR_ARG;
  const dim3 grid(n_seqs, a.n_v, (a.e + 7) / 8);
  const int rpl = (a.d + 7) / 8;
#define GO(RPL)                                                                       \
  do {                                                                                \
    if (a.per_channel) delta_scan_kernel<RPL, true><<<grid, FG_WAVE, 0, stream>>>(a);  \
    else delta_scan_kernel<RPL, false><<<grid, FG_WAVE, 0, stream>>>(a);              \
  } while (0)
  if (rpl <= 4) GO(4);
  else if (rpl <= 8) GO(8);
  else if (rpl <= 12) GO(12);
  else if (rpl <= 16) GO(16);
  else if (rpl <= 24) GO(24);
  else if (rpl <= 32) GO(32);
  else GO(64);
#undef GO
  return fg_launch_status();
}

// ------------------------------------------------------------------ chunks
// Within a chunk let L_t = the sum of log g up to token t, and S0 the state it starts from.  The writes u_t obey
//   (I + A) U = diag(beta) V - diag(beta exp(L)) K S0,   A[t, s] = beta_t exp(L_t - L_s) k_t . k_s  (s < t),
// the outputs and the state behind the chunk of n tokens are
//   O = diag(exp(L)) Q S0 + M U,   M[t, s] = exp(L_t - L_s) q_t . k_s  (s <= t),
//   S = exp(L_n) S0 + K^T diag(exp(L_n - L)) U.
// delta_chunk_prepare makes T = (I + A)^-1 and M for every chunk and head side by side; delta_chunk_scan walks a
// sequence's chunks in order, a workgroup 16 value channels of a head.  All products are fp32
// (v_mfma_f32_16x16x4_f32); an operand's k index runs as 16 j + 4 (lane / 16) + i over the four products i of a block
// j, so that a lane reads its operands as float4 and a result (rows 4 (lane / 16) + i) is the next product's second
// operand as it is.  Tokens beyond a chunk's last have beta = 0 and change nothing.
//
// Decays per channel: L_t is a vector, exp(L_t - L_s) stands inside the products over the channels, and in
//   A[t, s] = beta_t sum_c k_t[c] k_s[c] exp(L_t[c] - L_s[c])
// it is split at the start r of the 16 tokens that hold t: k_t exp(L_t - L_r) meets k_s exp(L_r - L_s).  For s before r
// both factors are at most one.  Inside the 16 tokens the second one grows; while no channel fades by more than
// 2^-DC_SAFE there both stay far inside fp32, else those 16 x 16 sums are taken pair by pair with the difference in the
// exponent.  delta_channel_prepare also leaves the chunk's rows with their decays multiplied in,
//   Q exp(L), K exp(L), K exp(L_n - L) and exp(L_n),
// and the scan takes those in place of the rows and the numbers per token.
#define DC 64  // tokens of a chunk
#define DC_LD (DC + 4)

typedef float f32x4 __attribute__((ext_vector_type(4)));

struct DeltaChunks {
  const int* chunk_start;  // [n_chunks + 1] first flat tokens
  const int* seq_chunk;    // [n_seqs + 1] first chunk of each sequence
  float* T; float* M;      // [n_chunks, n_v, 64, 64]; blocks of 16 x 16 above the diagonal are not written
  float* L;                // [n_chunks, n_v, 64]; decays per channel: exp(L_n), [n_chunks, n_v, d]
  float* Qd; float* Kd; float* Ke;  // decays per channel: [n_chunks, n_v, 64, d]
};
#define DC_SAFE 86.f  // in powers of two
__device__ __forceinline__ float exp2_hw(float x) { return __builtin_amdgcn_exp2f(x); }

__device__ __forceinline__ f32x4 mfma4(const float4& x, const float4& y, f32x4 acc) {
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, y.x, acc, 0, 0, 0);
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, y.y, acc, 0, 0, 0);
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, y.z, acc, 0, 0, 0);
  return __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, y.w, acc, 0, 0, 0);
}

// T = (I + A)^-1 of a chunk, from the lower triangle A_s in LDS through T_s to memory; the whole workgroup, 4 waves.
__device__ __forceinline__ void chunk_inverse(const float (&A_s)[DC][DC_LD], float (&T_s)[DC][DC_LD], float* T) {
  const int lane = threadIdx.x % FG_WAVE, wave = threadIdx.x / FG_WAVE, g = lane >> 4, r16 = lane & 15;
  {  // the inverse of the diagonal block of this wave: a lane a column
    float x[16];
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      float v = t == r16 ? 1.f : 0.f;
#pragma unroll
      for (int s = 0; s < t; ++s) v -= A_s[16 * wave + t][16 * wave + s] * x[s];
      x[t] = v;
    }
    if (g == 0) {
#pragma unroll
      for (int t = 0; t < 16; ++t) T_s[16 * wave + t][16 * wave + r16] = x[t];
    }
  }
  __syncthreads();
  for (int i = wave + 1; i < 4; ++i) {  // block column `wave`, downwards: T_ij = -T_ii sum_k A_ik T_kj
    f32x4 y = {0.f, 0.f, 0.f, 0.f};
    for (int k = wave; k < i; ++k) {
      const float4 av = *(const float4*)&A_s[16 * i + r16][16 * k + 4 * g];
      const float4 tv = make_float4(T_s[16 * k + 4 * g][16 * wave + r16], T_s[16 * k + 4 * g + 1][16 * wave + r16],
                                    T_s[16 * k + 4 * g + 2][16 * wave + r16], T_s[16 * k + 4 * g + 3][16 * wave + r16]);
      y = mfma4(av, tv, y);
    }
    const float4 tii = *(const float4*)&T_s[16 * i + r16][16 * i + 4 * g];
    const f32x4 res = mfma4(tii, make_float4(-y[0], -y[1], -y[2], -y[3]), f32x4{0.f, 0.f, 0.f, 0.f});
#pragma unroll
    for (int r = 0; r < 4; ++r) T_s[16 * i + 4 * g + r][16 * wave + r16] = res[r];
  }
  __syncthreads();
  for (int e = threadIdx.x; e < DC * DC / 4; e += 256) {
    const int t = e / (DC / 4), s = 4 * (e % (DC / 4));
    if (s / 16 <= t / 16) *(float4*)(T + t * DC + s) = *(const float4*)&T_s[t][s];
  }
}

// grid (n_chunks, n_v), 4 waves; NDM >= d / 16
template <int NDM>
__global__ __launch_bounds__(256) void delta_chunk_prepare_kernel(const DeltaScanArgs a, const DeltaChunks ch) {
  __shared__ __attribute__((aligned(16))) float A_s[DC][DC_LD], T_s[DC][DC_LD];
  __shared__ float L_s[DC], beta_s[DC];
  const int lane = threadIdx.x % FG_WAVE, wave = threadIdx.x / FG_WAVE, g = lane >> 4, r16 = lane & 15;
  const int c = blockIdx.x, h = blockIdx.y, hq = h / (a.n_v / a.n_qk), nd = a.d / 16;
  const int t0 = ch.chunk_start[c], n = ch.chunk_start[c + 1] - t0;
  const int k_col = a.n_qk * a.d, b_col = 2 * k_col + a.n_v * a.e + h;
  const size_t at = (size_t)c * a.n_v + h;
  if (wave == 0) {
    const float* row = a.rows + (size_t)(t0 + min(lane, n - 1)) * a.stride;
    float L = lane < n ? row[a.g_col + h] : 0.f;
#pragma unroll
    for (int m = 1; m < DC; m <<= 1) {
      const float o = __shfl_up(L, m, FG_WAVE);
      if (lane >= m) L += o;
    }
    L_s[lane] = L;
    beta_s[lane] = lane < n ? row[b_col] : 0.f;
    ch.L[at * DC + lane] = L;
  }
  __syncthreads();
  float4 kf[NDM], qf[NDM];
  {
    const float* row = a.rows + (size_t)(t0 + min(16 * wave + r16, n - 1)) * a.stride + hq * a.d + 4 * g;
#pragma unroll
    for (int j = 0; j < NDM; ++j) {
      if (j < nd) {  // uniform
        qf[j] = *(const float4*)(row + 16 * j);
        kf[j] = *(const float4*)(row + k_col + 16 * j);
      }
    }
  }
  for (int b = 0; b <= wave; ++b) {
    const float* row = a.rows + (size_t)(t0 + min(16 * b + r16, n - 1)) * a.stride + k_col + hq * a.d + 4 * g;
    f32x4 kk = {0.f, 0.f, 0.f, 0.f}, qk = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < NDM; ++j) {
      if (j < nd) {
        const float4 o = *(const float4*)(row + 16 * j);
        kk = mfma4(kf[j], o, kk);
        qk = mfma4(qf[j], o, qk);
      }
    }
    const int s = 16 * b + r16;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = 16 * wave + 4 * g + i;
      const float dec = expf(L_s[t] - L_s[s]);  // (not used above the diagonal)
      A_s[t][s] = s < t ? beta_s[t] * dec * kk[i] : 0.f;
      ch.M[at * DC * DC + t * DC + s] = s <= t ? dec * qk[i] : 0.f;
    }
  }
  __syncthreads();
  chunk_inverse(A_s, T_s, ch.T + at * DC * DC);
}

// Decays per channel: grid (n_chunks, n_v), 4 waves, wave w the tokens 16 w ..; NDM >= d / 16.  LDS: P[t][c] = the sum of
// log2 g[c] from the start of t's 16 tokens up to t (base 2: the hardware's exponential takes it as it is).
template <int NDM>
__global__ __launch_bounds__(256) void delta_channel_prepare_kernel(const DeltaScanArgs a, const DeltaChunks ch) {
  constexpr int LD = 16 * NDM + 4;
  __shared__ __attribute__((aligned(16))) float A_s[DC][DC_LD], T_s[DC][DC_LD];
  __shared__ __attribute__((aligned(16))) float P_s[DC][LD];
  __shared__ float beta_s[DC];
  const int lane = threadIdx.x % FG_WAVE, wave = threadIdx.x / FG_WAVE, g = lane >> 4, r16 = lane & 15;
  const int c = blockIdx.x, h = blockIdx.y, d = a.d, hq = h / (a.n_v / a.n_qk), nd = d / 16;
  const int t0 = ch.chunk_start[c], n = ch.chunk_start[c + 1] - t0;
  const int k_col = a.n_qk * d, b_col = 2 * k_col + a.n_v * a.e + h, g_col = a.g_col + h * d;
  const size_t at = (size_t)c * a.n_v + h;
  for (int i = threadIdx.x; i < 4 * d; i += 256) {  // a thread a channel of 16 tokens
    const int j = i / d, k = i % d;
    float x[16], sum = 0.f;
#pragma unroll
    for (int t = 0; t < 16; ++t) x[t] = a.rows[(size_t)(t0 + min(16 * j + t, n - 1)) * a.stride + g_col + k];
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      sum += 16 * j + t < n ? x[t] * 1.4426950408889634f : 0.f;
      P_s[16 * j + t][k] = sum;
    }
  }
  if (wave == 0) beta_s[lane] = lane < n ? a.rows[(size_t)(t0 + min(lane, n - 1)) * a.stride + b_col] : 0.f;
  __syncthreads();
  // this wave's 16 tokens as first operands, with exp(P) multiplied in (what meets earlier tokens)
  const int t_row = 16 * wave + r16;
  const bool t_in = t_row < n;
  float4 kf[NDM], qf[NDM];
  bool safe = true;
  {
    const float* row = a.rows + (size_t)(t0 + min(t_row, n - 1)) * a.stride + hq * d + 4 * g;
    float* qd = ch.Qd + (at * DC + t_row) * d + 4 * g;
    float* kd = ch.Kd + (at * DC + t_row) * d + 4 * g;
    float* ke = ch.Ke + (at * DC + t_row) * d + 4 * g;
#pragma unroll
    for (int j = 0; j < NDM; ++j) {
      if (j < nd) {  // uniform
        const float4 q = *(const float4*)(row + 16 * j), k = *(const float4*)(row + k_col + 16 * j);
        const int col = 16 * j + 4 * g;
        const float4 P = *(const float4*)&P_s[t_row][col];
        float4 own = *(const float4*)&P_s[16 * wave + 15][col];
        float4 before = make_float4(0.f, 0.f, 0.f, 0.f), behind = before;
#pragma unroll
        for (int m = 0; m < 4; ++m) {
          const float4 x = *(const float4*)&P_s[16 * m + 15][col];
          if (m < wave) { before.x += x.x; before.y += x.y; before.z += x.z; before.w += x.w; }
          if (m > wave) { behind.x += x.x; behind.y += x.y; behind.z += x.z; behind.w += x.w; }
        }
        safe = safe && fminf(fminf(own.x, own.y), fminf(own.z, own.w)) > -DC_SAFE;
        const float4 eP = make_float4(exp2_hw(P.x), exp2_hw(P.y), exp2_hw(P.z), exp2_hw(P.w));
        const float4 eb = make_float4(exp2_hw(before.x), exp2_hw(before.y), exp2_hw(before.z), exp2_hw(before.w));
        const float4 ee = make_float4(exp2_hw(own.x - P.x + behind.x), exp2_hw(own.y - P.y + behind.y), exp2_hw(own.z - P.z + behind.z),
                                      exp2_hw(own.w - P.w + behind.w));
        qf[j] = make_float4(q.x * eP.x, q.y * eP.y, q.z * eP.z, q.w * eP.w);
        kf[j] = make_float4(k.x * eP.x, k.y * eP.y, k.z * eP.z, k.w * eP.w);
        const float in = t_in ? 1.f : 0.f;
        *(float4*)(qd + 16 * j) = make_float4(in * qf[j].x * eb.x, in * qf[j].y * eb.y, in * qf[j].z * eb.z, in * qf[j].w * eb.w);
        *(float4*)(kd + 16 * j) = make_float4(in * kf[j].x * eb.x, in * kf[j].y * eb.y, in * kf[j].z * eb.z, in * kf[j].w * eb.w);
        *(float4*)(ke + 16 * j) = make_float4(in * k.x * ee.x, in * k.y * ee.y, in * k.z * ee.z, in * k.w * ee.w);
        if (wave == 3 && r16 == 15)
          *(float4*)(ch.L + at * d + col) = make_float4(eb.x * exp2_hw(own.x), eb.y * exp2_hw(own.y), eb.z * exp2_hw(own.z), eb.w * exp2_hw(own.w));
      }
    }
  }
  safe = __all(safe);
  for (int b = 0; b <= wave; ++b) {
    const float* row = a.rows + (size_t)(t0 + min(16 * b + r16, n - 1)) * a.stride + k_col + hq * d;
    f32x4 kk = {0.f, 0.f, 0.f, 0.f}, qk = {0.f, 0.f, 0.f, 0.f};
    if (b < wave || safe) {  // uniform in the wave
#pragma unroll
      for (int j = 0; j < NDM; ++j) {
        if (j < nd) {
          const int col = 16 * j + 4 * g;
          float4 o = *(const float4*)(row + col);
          const float4 P = *(const float4*)&P_s[16 * b + r16][col];
          float4 x = make_float4(-P.x, -P.y, -P.z, -P.w);
          for (int m = b; m < wave; ++m) {  // up to the start of this wave's tokens
            const float4 y = *(const float4*)&P_s[16 * m + 15][col];
            x.x += y.x; x.y += y.y; x.z += y.z; x.w += y.w;
          }
          o.x *= exp2_hw(x.x); o.y *= exp2_hw(x.y); o.z *= exp2_hw(x.z); o.w *= exp2_hw(x.w);
          kk = mfma4(kf[j], o, kk);
          qk = mfma4(qf[j], o, qk);
        }
      }
    } else {  // a lane the pairs (4 g + i, r16) of the wave's own tokens, channel by channel
      const float* tr[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) tr[i] = a.rows + (size_t)(t0 + min(16 * wave + 4 * g + i, n - 1)) * a.stride + hq * d;
      for (int k = 0; k < d; ++k) {
        const float ks = row[k], Ps = P_s[16 * wave + r16][k];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float f = ks * exp2_hw(fminf(P_s[16 * wave + 4 * g + i][k] - Ps, 0.f));  // (pairs with t < s are not used)
          kk[i] = fmaf(tr[i][k_col + k], f, kk[i]);
          qk[i] = fmaf(tr[i][k], f, qk[i]);
        }
      }
    }
    const int s = 16 * b + r16;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = 16 * wave + 4 * g + i;
      A_s[t][s] = s < t ? beta_s[t] * kk[i] : 0.f;
      ch.M[at * DC * DC + t * DC + s] = s <= t ? qk[i] : 0.f;
    }
  }
  __syncthreads();
  chunk_inverse(A_s, T_s, ch.T + at * DC * DC);
}

// grid (n_seqs, n_v, ceil(e / 16)), 4 waves: wave w takes tokens 16 w .. of a chunk, and the key channels of the
// blocks w, w + 4, .. of the state.  CH: decays per channel, operands from delta_channel_prepare.
template <int NDM, bool CH>
__global__ __launch_bounds__(256) void delta_chunk_scan_kernel(const DeltaScanArgs a, const DeltaChunks ch) {
  constexpr int NT = (NDM + 3) / 4;
  __shared__ __attribute__((aligned(16))) float S_s[16][16 * NDM + 4];             // the state, by value channel
  __shared__ __attribute__((aligned(16))) float X_s[16][DC_LD], U_s[16][DC_LD], D_s[16][DC_LD];
  const int lane = threadIdx.x % FG_WAVE, wave = threadIdx.x / FG_WAVE, g = lane >> 4, r16 = lane & 15;
  const int b = blockIdx.x, h = blockIdx.y, col = blockIdx.z * 16 + r16;
  const bool col_ok = col < a.e;
  const int d = a.d, e = a.e, nd = d / 16, hq = h / (a.n_v / a.n_qk);
  const int k_col = a.n_qk * d, v_col = 2 * k_col + h * e + min(col, e - 1), b_col = 2 * k_col + a.n_v * e + h;
  float* S_mem = a.state + (size_t)a.slot_ids[b] * a.slot_stride + (size_t)h * d * e;
  f32x4 S[NT];
#pragma unroll
  for (int m = 0; m < NT; ++m) {
    const int ti = wave + 4 * m;
#pragma unroll
    for (int i = 0; i < 4; ++i) S[m][i] = ti < nd && col_ok ? S_mem[(size_t)(16 * ti + 4 * g + i) * e + col] : 0.f;
    if (ti < nd) *(f32x4*)&S_s[r16][16 * ti + 4 * g] = S[m];
  }
  const int c_end = ch.seq_chunk[b + 1];
  float4 kf[NDM], qf[NDM];
  auto ask_rows = [&](int c) {  // this wave's 16 tokens of chunk c as first operands
    const int t0 = ch.chunk_start[c], n = ch.chunk_start[c + 1] - t0;
    const size_t own = (((size_t)c * a.n_v + h) * DC + 16 * wave + r16) * d + 4 * g;
    const float* row = a.rows + (size_t)(t0 + min(16 * wave + r16, n - 1)) * a.stride + hq * d + 4 * g;
    const float* qrow = CH ? ch.Qd + own : row;
    const float* krow = CH ? ch.Kd + own : row + k_col;
#pragma unroll
    for (int j = 0; j < NDM; ++j) {
      if (j < nd) {  // uniform
        qf[j] = *(const float4*)(qrow + 16 * j);
        kf[j] = *(const float4*)(krow + 16 * j);
      }
    }
  };
  int c = ch.seq_chunk[b];
  if (c < c_end) ask_rows(c);
  for (; c < c_end; ++c) {
    const int t0 = ch.chunk_start[c], n = ch.chunk_start[c + 1] - t0;
    const size_t at = (size_t)c * a.n_v + h;
    // what the later phases need, asked for now
    float4 tf[4], mf[4];
    const float* t_row = ch.T + at * DC * DC + (size_t)(16 * wave + r16) * DC + 4 * g;
    const float* m_row = ch.M + at * DC * DC + (size_t)(16 * wave + r16) * DC + 4 * g;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      if (j <= wave) {  // uniform in the wave
        tf[j] = *(const float4*)(t_row + 16 * j);
        mf[j] = *(const float4*)(m_row + 16 * j);
      }
    }
    float beta[4], eL[4], eD[4], v[4];
    const float L_end = CH ? 0.f : ch.L[at * DC + DC - 1];
    f32x4 keep[NT];  // what is left of each of this wave's state rows behind the chunk
    if (CH) {
#pragma unroll
      for (int m = 0; m < NT; ++m)
        if (wave + 4 * m < nd) keep[m] = *(const f32x4*)(ch.L + at * d + 16 * (wave + 4 * m) + 4 * g);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = 16 * wave + 4 * g + i;
      const float L = CH ? 0.f : ch.L[at * DC + t];
      const float* row = a.rows + (size_t)(t0 + min(t, n - 1)) * a.stride;
      beta[i] = t < n ? row[b_col] : 0.f;
      v[i] = row[v_col];
      eL[i] = expf(L);
      eD[i] = expf(L_end - L);
    }
    __syncthreads();  // S_s is complete
    // ---- 1. X = beta (V - exp(L) K S), and exp(L) Q S
    f32x4 ks = {0.f, 0.f, 0.f, 0.f}, o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < NDM; ++j) {
      if (j < nd) {
        const float4 sv = *(const float4*)&S_s[r16][16 * j + 4 * g];
        ks = mfma4(kf[j], sv, ks);
        o = mfma4(qf[j], sv, o);
      }
    }
    if (c + 1 < c_end) ask_rows(c + 1);
    // the chunk's keys as first operands of K^T U: channel 16 ti + r16, token 16 j + 4 g + i
    float kt[NT][4][4];
#pragma unroll
    for (int m = 0; m < NT; ++m) {
      if (wave + 4 * m < nd) {
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
          for (int i = 0; i < 4; ++i)
            kt[m][j][i] = CH ? ch.Ke[(at * DC + 16 * j + 4 * g + i) * d + 16 * (wave + 4 * m) + r16]
                             : a.rows[(size_t)(t0 + min(16 * j + 4 * g + i, n - 1)) * a.stride + k_col + hq * d +
                                      16 * (wave + 4 * m) + r16];
      }
    }
    f32x4 x;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      x[i] = beta[i] * (v[i] - eL[i] * ks[i]);
      o[i] *= eL[i];
    }
    *(f32x4*)&X_s[r16][16 * wave + 4 * g] = x;
    __syncthreads();
    // ---- 2. U = T X
    f32x4 u = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j <= wave) u = mfma4(tf[j], *(const float4*)&X_s[r16][16 * j + 4 * g], u);
    *(f32x4*)&U_s[r16][16 * wave + 4 * g] = u;
#pragma unroll
    for (int i = 0; i < 4; ++i) u[i] *= eD[i];
    *(f32x4*)&D_s[r16][16 * wave + 4 * g] = u;
    __syncthreads();
    // ---- 3. O = exp(L) Q S + M U
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j <= wave) o = mfma4(mf[j], *(const float4*)&U_s[r16][16 * j + 4 * g], o);
    if (col_ok) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = 16 * wave + 4 * g + i;
        if (t < n) a.out[(size_t)(t0 + t) * ((size_t)a.n_v * e) + h * e + col] = o[i];
      }
    }
    // ---- 4. S = exp(L_n) S + K^T diag(exp(L_n - L)) U
    const float all = CH ? 1.f : expf(L_end);
#pragma unroll
    for (int m = 0; m < NT; ++m) {
      const int ti = wave + 4 * m;
      if (ti < nd) {
        if (CH) S[m] *= keep[m];
        else S[m] *= all;
#pragma unroll
        for (int j = 0; j < 4; ++j)
          S[m] = mfma4(make_float4(kt[m][j][0], kt[m][j][1], kt[m][j][2], kt[m][j][3]), *(const float4*)&D_s[r16][16 * j + 4 * g], S[m]);
        *(f32x4*)&S_s[r16][16 * ti + 4 * g] = S[m];  // (everybody has read the old state: two barriers ago)
      }
    }
  }
#pragma unroll
  for (int m = 0; m < NT; ++m) {
    const int ti = wave + 4 * m;
    if (ti < nd && col_ok) {
#pragma unroll
      for (int i = 0; i < 4; ++i) S_mem[(size_t)(16 * ti + 4 * g + i) * e + col] = S[m][i];
    }
  }
}

extern "C" int fg_delta_chunk_tokens() { return DC; }

// d a multiple of 16 up to 256, rows 16-byte aligned
extern "C" int fg_delta_chunk_scan(const DeltaScanArgs* args, const DeltaChunks* chunks, int n_chunks, int n_seqs,
                                   hipStream_t stream) {
  if (n_seqs <= 0 || n_chunks <= 0) return FG_OK;
  const DeltaScanArgs& a = *args;
  const DeltaChunks& ch = *chunks;
  if (!delta_scan_ok(a, n_seqs) || a.d % 16 || a.d > 256 || a.stride % 4 || ((uintptr_t)a.rows & 15) || n_chunks > 2147483647 / 64 ||
      !ch.chunk_start || !ch.seq_chunk || !ch.T || !ch.M || !ch.L || (a.per_channel && (!ch.Qd || !ch.Kd || !ch.Ke)))
    return FG_ERR_ARG;
  const dim3 pgrid(n_chunks, a.n_v), sgrid(n_seqs, a.n_v, (a.e + 15) / 16);
#define GO(NDM)                                                               \
  do {                                                                        \
    if (a.per_channel) {                                                      \
      delta_channel_prepare_kernel<NDM><<<pgrid, 256, 0, stream>>>(a, ch);    \
      delta_chunk_scan_kernel<NDM, true><<<sgrid, 256, 0, stream>>>(a, ch);   \
    } else {                                                                  \
      delta_chunk_prepare_kernel<NDM><<<pgrid, 256, 0, stream>>>(a, ch);      \
      delta_chunk_scan_kernel<NDM, false><<<sgrid, 256, 0, stream>>>(a, ch);  \
    }                                                                         \
  } while (0)
  if (a.d <= 64) GO(4);
  else if (a.d <= 128) GO(8);
  else GO(16);
#undef GO
  return fg_launch_status();
}
