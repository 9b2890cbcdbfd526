// Linear attention whose state fades by a constant per head: per head, with S [d, e] in fp32 kept per request,
//
//   S_t = a S_(t-1) + k_t v_t^T;   o_t = S_t^T q_t;   q, k, v = silu of a product's columns
//
//  lightning_scan    token by token: a wave eight value channels of a head, as in delta_rule.hip (decoded tokens, short
//                    portions).
//  lightning_chunk_* long runs of tokens, 64 at a time as matrix products, all chunks side by side.  With n tokens in a
//                    chunk, S0 the state it starts from, t and s counted from its first token:
//                      states    a chunk's own contribution   C = sum_s a^(n-1-s) k_s v_s^T
//                      combine   per sequence, chunk after chunk, element by element: S0 of each chunk; S <- a^n S + C
//                      outputs   O = diag(a^(t+1)) Q S0 + M V,   M[t, s] = a^(t-s) q_t . k_s  (s <= t)
//                    Products are fp32 (v_mfma_f32_16x16x4_f32; an operand's k index runs as 16 j + 4 (lane / 16) + i over
//                    the four products i of a block j): the same as token by token within rounding.
#include "common.h"

#define LC 64  // tokens of a chunk
#define LC_LD (LC + 4)
#define LC_COLS 128  // value channels a workgroup takes

typedef float f32x4 __attribute__((ext_vector_type(4)));

struct LightningArgs {
  const float* rows; int stride, q_col, k_col, v_col;  // fp32 rows: H heads of d, of d, of e
  int H, d, e;
  const float* log_decay;                 // [H]
  float* state; long long slot_stride;    // S of slot s, head h at s * slot_stride + h * d * e
  const int* slot_ids; const int* q_start;
  float* out;                             // [T, H * e]
};
struct LightningChunks {
  const int* chunk_start;  // [n_chunks + 1] first flat tokens
  const int* seq_chunk;    // [n_seqs + 1] first chunk of each sequence
  float* states;           // [n_chunks, H, d, e]
};

// (the hardware's exponential and reciprocal: a few ulp of 32-bit)
__device__ __forceinline__ float lt_silu(float x) { return x * __builtin_amdgcn_rcpf(1.f + __expf(-x)); }
__device__ __forceinline__ float4 lt_silu4(const float4& x) { return make_float4(lt_silu(x.x), lt_silu(x.y), lt_silu(x.z), lt_silu(x.w)); }
__device__ __forceinline__ f32x4 lt_mfma4(const float4& x, const float4& y, f32x4 acc) {
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, y.x, acc, 0, 0, 0);
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, y.y, acc, 0, 0, 0);
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, y.z, acc, 0, 0, 0);
  return __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, y.w, acc, 0, 0, 0);
}
// the sum over the eight lanes that hold a column (equal lane % 8), in each of them
__device__ __forceinline__ float lt_column_sum(float v) {
  v += __uint_as_float(__builtin_amdgcn_update_dpp(0, __float_as_uint(v), 0x128 /* row_ror:8 */, 0xf, 0xf, false));
  const auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  v = __uint_as_float(a[0]) + __uint_as_float(a[1]);
  const auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  return __uint_as_float(b[0]) + __uint_as_float(b[1]);
}

// ------------------------------------------------------------ token by token
#define LT_TOKENS_FOR(RPL) ((RPL) <= 16 ? 8 : 4)  // tokens staged at a time

// grid (B, H, ceil(e / 8)), one wave: lane l holds column l & 7 and the key channels rg * rpl .. (rg = l >> 3) of it.
template <int RPL>
__global__ __launch_bounds__(FG_WAVE) void lightning_scan_kernel(const LightningArgs a) {
  constexpr int RUN = LT_TOKENS_FOR(RPL), NJ = (RPL + 7) / 8;
  // [RUN][2][8 parts of RPL + 4]: k, q; key channel r of part p = r / rpl at p * (RPL + 4) + r % rpl, zeros behind rpl
  constexpr int PS = RPL + 4, VS = 8 * PS;
  __shared__ __attribute__((aligned(16))) float lds[RUN * 2 * VS];
  const int lane = threadIdx.x, b = blockIdx.x, h = blockIdx.y;
  const int rg = lane >> 3, col = blockIdx.z * 8 + (lane & 7);
  const bool col_ok = col < a.e;
  const int d = a.d, e = a.e, rpl = (d + 7) / 8, r0 = rg * rpl;
  const int t_begin = a.q_start[b], t_end = a.q_start[b + 1];
  if (t_begin >= t_end) return;  // uniform
  const float decay = expf(a.log_decay[h]);
  float* S_mem = a.state + (size_t)a.slot_ids[b] * a.slot_stride + (size_t)h * d * e;
  float S[RPL];
#pragma unroll
  for (int i = 0; i < RPL; ++i) S[i] = (i < rpl && r0 + i < d && col_ok) ? S_mem[(size_t)(r0 + i) * e + col] : 0.f;
  for (int i = lane; i < RUN * 2 * VS; i += FG_WAVE) lds[i] = 0.f;
  int src[NJ], dst[NJ];
  bool mine[NJ];
#pragma unroll
  for (int j = 0; j < NJ; ++j) {
    const int r = lane + FG_WAVE * j;
    mine[j] = r < d;
    src[j] = h * d + min(r, d - 1);
    dst[j] = (r / rpl) * PS + r % rpl;
  }
  const int v_src = a.v_col + h * e + min(col, e - 1);
  float pk[RUN][NJ], pq[RUN][NJ], pv[RUN];
  auto fetch = [&](int t0) {
#pragma unroll
    for (int tt = 0; tt < RUN; ++tt) {
      const float* row = a.rows + (size_t)min(t0 + tt, t_end - 1) * a.stride;
#pragma unroll
      for (int j = 0; j < NJ; ++j) {
        pk[tt][j] = row[a.k_col + src[j]];
        pq[tt][j] = row[a.q_col + src[j]];
      }
      pv[tt] = row[v_src];
    }
  };
  fetch(t_begin);
  for (int t0 = t_begin; t0 < t_end; t0 += RUN) {
    const int n = min(RUN, t_end - t0);
    __syncthreads();  // the run before has been read
    float v[RUN];
#pragma unroll
    for (int tt = 0; tt < RUN; ++tt) {
      v[tt] = lt_silu(pv[tt]);
      if (tt < n) {  // uniform
#pragma unroll
        for (int j = 0; j < NJ; ++j) {
          if (mine[j]) {
            lds[tt * 2 * VS + dst[j]] = lt_silu(pk[tt][j]);
            lds[tt * 2 * VS + VS + dst[j]] = lt_silu(pq[tt][j]);
          }
        }
      }
    }
    __syncthreads();
    if (t0 + RUN < t_end) fetch(t0 + RUN);  // in flight while this run is computed
    float acc[RUN];
#pragma unroll
    for (int tt = 0; tt < RUN; ++tt) {
      float part[4] = {0.f, 0.f, 0.f, 0.f};
      if (tt < n) {  // uniform
        const float4* kp = (const float4*)(lds + tt * 2 * VS + rg * PS);
        const float4* qp = (const float4*)(lds + tt * 2 * VS + VS + rg * PS);
#pragma unroll
        for (int i4 = 0; i4 < RPL / 4; ++i4) {
          const float4 k4 = kp[i4], q4 = qp[i4];
          const float kk[4] = {k4.x, k4.y, k4.z, k4.w}, qq[4] = {q4.x, q4.y, q4.z, q4.w};
#pragma unroll
          for (int u = 0; u < 4; ++u) {
            S[4 * i4 + u] = decay * S[4 * i4 + u] + kk[u] * v[tt];
            part[u] += S[4 * i4 + u] * qq[u];
          }
        }
      }
      acc[tt] = (part[0] + part[1]) + (part[2] + part[3]);
    }
#pragma unroll
    for (int tt = 0; tt < RUN; ++tt) acc[tt] = lt_column_sum(acc[tt]);
    if (rg == 0 && col_ok) {
#pragma unroll
      for (int tt = 0; tt < RUN; ++tt)
        if (tt < n) a.out[(size_t)(t0 + tt) * ((size_t)a.H * e) + h * e + col] = acc[tt];
    }
  }
#pragma unroll
  for (int i = 0; i < RPL; ++i)
    if (i < rpl && r0 + i < d && col_ok) S_mem[(size_t)(r0 + i) * e + col] = S[i];
}

static bool lightning_ok(const LightningArgs& a, int n_seqs) {
  return a.H > 0 && a.H <= 65535 && a.d > 0 && a.d <= 512 && a.e > 0 && (a.e + 7) / 8 <= 65535 && n_seqs <= 2147483647 && a.rows &&
         a.log_decay && a.state && a.slot_ids && a.q_start && a.out && a.q_col >= 0 && a.k_col >= 0 && a.v_col >= 0 &&
         a.q_col + a.H * a.d <= a.stride && a.k_col + a.H * a.d <= a.stride && a.v_col + a.H * a.e <= a.stride;
}

extern "C" int fg_lightning_scan(const LightningArgs* args, int n_seqs, hipStream_t stream) {
  if (n_seqs <= 0) return FG_OK;
  const LightningArgs& a = *args;
  if (!lightning_ok(a, n_seqs)) return FG_ERR_ARG;
  const dim3 grid(n_seqs, a.H, (a.e + 7) / 8);
  const int rpl = (a.d + 7) / 8;
#define GO(RPL) lightning_scan_kernel<RPL><<<grid, FG_WAVE, 0, stream>>>(a)
  if (rpl <= 4) GO(4);
  else if (rpl <= 8) GO(8);
  else if (rpl <= 16) GO(16);
  else if (rpl <= 32) GO(32);
  else GO(64);
#undef GO
  return fg_launch_status();
}

// -------------------------------------------------------------------- chunks
// grid (n_chunks, H, ceil(e / 128)), 4 waves; wave w the state's rows of the blocks w, w + 4, .. of 16 key channels.
template <int NDM>
__global__ __launch_bounds__(256) void lightning_chunk_states_kernel(const LightningArgs a, const LightningChunks ch) {
  constexpr int NT = (NDM + 3) / 4;
  __shared__ float V_s[LC][LC_COLS + 4];
  const int lane = threadIdx.x % FG_WAVE, wave = threadIdx.x / FG_WAVE, g = lane >> 4, r16 = lane & 15;
  const int c = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * LC_COLS, nd = a.d / 16, cols = min(LC_COLS, a.e - c0);
  const int t0 = ch.chunk_start[c], n = ch.chunk_start[c + 1] - t0;
  const float lg = a.log_decay[h];
  float kt[NT][4][4];
#pragma unroll
  for (int m = 0; m < NT; ++m) {
    if (wave + 4 * m < nd) {  // uniform in the wave
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i)
          kt[m][j][i] = a.rows[(size_t)(t0 + min(16 * j + 4 * g + i, n - 1)) * a.stride + a.k_col + h * a.d + 16 * (wave + 4 * m) + r16];
    }
  }
  {
    const int col = threadIdx.x % LC_COLS, t_own = threadIdx.x / LC_COLS;  // two tokens at a time
    const float* vp = a.rows + a.v_col + h * a.e + c0 + min(col, cols - 1);
#pragma unroll
    for (int u0 = 0; u0 < LC / 2; u0 += 16) {
      float v[16];
#pragma unroll
      for (int u = 0; u < 16; ++u) v[u] = vp[(size_t)(t0 + min(2 * (u0 + u) + t_own, n - 1)) * a.stride];
#pragma unroll
      for (int u = 0; u < 16; ++u) V_s[2 * (u0 + u) + t_own][col] = lt_silu(v[u]);
    }
  }
  float fade[4][4];
#pragma unroll
  for (int j = 0; j < 4; ++j)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int s = 16 * j + 4 * g + i;
      fade[j][i] = s < n ? expf(lg * (float)(n - 1 - s)) : 0.f;
    }
#pragma unroll
  for (int m = 0; m < NT; ++m)
    if (wave + 4 * m < nd) {
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) kt[m][j][i] = lt_silu(kt[m][j][i]) * fade[j][i];
    }
  __syncthreads();
  float* out = ch.states + ((size_t)c * a.H + h) * a.d * a.e + c0;
  for (int cb = 0; 16 * cb < cols; ++cb) {
    float4 v[4];
#pragma unroll
    for (int j = 0; j < 4; ++j)
      v[j] = make_float4(V_s[16 * j + 4 * g][16 * cb + r16], V_s[16 * j + 4 * g + 1][16 * cb + r16],
                         V_s[16 * j + 4 * g + 2][16 * cb + r16], V_s[16 * j + 4 * g + 3][16 * cb + r16]);
#pragma unroll
    for (int m = 0; m < NT; ++m) {
      const int ti = wave + 4 * m;
      if (ti < nd) {
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < 4; ++j) acc = lt_mfma4(make_float4(kt[m][j][0], kt[m][j][1], kt[m][j][2], kt[m][j][3]), v[j], acc);
        if (16 * cb + r16 < cols) {
#pragma unroll
          for (int i = 0; i < 4; ++i) out[(size_t)(16 * ti + 4 * g + i) * a.e + 16 * cb + r16] = acc[i];
        }
      }
    }
  }
}

// grid (ceil(d * e / 256), H, n_seqs), a thread an element of the state: `states` leaves with what each chunk starts from
#define LC_AHEAD 8
__global__ __launch_bounds__(256) void lightning_combine_kernel(const LightningArgs a, const LightningChunks ch) {
  const int h = blockIdx.y, b = blockIdx.z, per = a.d * a.e;
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i >= per) return;
  const float lg = a.log_decay[h];
  float* S_mem = a.state + (size_t)a.slot_ids[b] * a.slot_stride + (size_t)h * per + i;
  float S = *S_mem;
  const int c_begin = ch.seq_chunk[b], c_end = ch.seq_chunk[b + 1];
  const size_t step = (size_t)a.H * per;
  for (int c = c_begin; c < c_end; c += LC_AHEAD) {
    float* at = ch.states + ((size_t)c * a.H + h) * per + i;
    float add[LC_AHEAD], keep[LC_AHEAD];
#pragma unroll
    for (int j = 0; j < LC_AHEAD; ++j) {
      const int cc = min(c + j, c_end - 1);
      add[j] = at[(size_t)(cc - c) * step];
      keep[j] = expf(lg * (float)(ch.chunk_start[cc + 1] - ch.chunk_start[cc]));
    }
#pragma unroll
    for (int j = 0; j < LC_AHEAD; ++j) {
      if (c + j < c_end) {  // uniform
        at[(size_t)j * step] = S;
        S = keep[j] * S + add[j];
      }
    }
  }
  *S_mem = S;
}

// grid (n_chunks, H, ceil(e / 128)), 4 waves: M by rows (wave w the tokens 16 w ..), then each wave blocks of 16 value
// channels for all 64 tokens.
template <int NDM>
__global__ __launch_bounds__(256) void lightning_chunk_out_kernel(const LightningArgs a, const LightningChunks ch) {
  __shared__ __attribute__((aligned(16))) float Q_s[LC][16 * NDM + 4];
  __shared__ __attribute__((aligned(16))) float M_s[LC][LC_LD];
  const int lane = threadIdx.x % FG_WAVE, wave = threadIdx.x / FG_WAVE, g = lane >> 4, r16 = lane & 15;
  const int c = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * LC_COLS, d = a.d, nd = d / 16, cols = min(LC_COLS, a.e - c0);
  const int t0 = ch.chunk_start[c], n = ch.chunk_start[c + 1] - t0;
  const float lg = a.log_decay[h];
  {
    float4 qf[NDM];
    const float* row = a.rows + (size_t)(t0 + min(16 * wave + r16, n - 1)) * a.stride + a.q_col + h * d + 4 * g;
#pragma unroll
    for (int j = 0; j < NDM; ++j)
      if (j < nd) qf[j] = *(const float4*)(row + 16 * j);  // uniform
#pragma unroll
    for (int j = 0; j < NDM; ++j)
      if (j < nd) {
        qf[j] = lt_silu4(qf[j]);
        *(float4*)&Q_s[16 * wave + r16][16 * j + 4 * g] = qf[j];
      }
    for (int b = 0; b <= wave; ++b) {
      const float* krow = a.rows + (size_t)(t0 + min(16 * b + r16, n - 1)) * a.stride + a.k_col + h * d + 4 * g;
      f32x4 qk = {0.f, 0.f, 0.f, 0.f};
      float4 kf[NDM];
#pragma unroll
      for (int j = 0; j < NDM; ++j)
        if (j < nd) kf[j] = *(const float4*)(krow + 16 * j);
#pragma unroll
      for (int j = 0; j < NDM; ++j)
        if (j < nd) qk = lt_mfma4(qf[j], lt_silu4(kf[j]), qk);
      const int s = 16 * b + r16;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = 16 * wave + 4 * g + i;
        M_s[t][s] = s <= t && t < n ? expf(lg * (float)(t - s)) * qk[i] : 0.f;
      }
    }
  }
  __syncthreads();
  const float* S0 = ch.states + ((size_t)c * a.H + h) * d * a.e + c0;
  for (int cb = wave; 16 * cb < cols; cb += 4) {
    const int col = min(16 * cb + r16, cols - 1);
    f32x4 acc[4];
#pragma unroll
    for (int tb = 0; tb < 4; ++tb) acc[tb] = f32x4{0.f, 0.f, 0.f, 0.f};
    float4 v[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const float* vp = a.rows + a.v_col + h * a.e + c0 + col;
      v[j] = make_float4(vp[(size_t)(t0 + min(16 * j + 4 * g, n - 1)) * a.stride], vp[(size_t)(t0 + min(16 * j + 4 * g + 1, n - 1)) * a.stride],
                         vp[(size_t)(t0 + min(16 * j + 4 * g + 2, n - 1)) * a.stride], vp[(size_t)(t0 + min(16 * j + 4 * g + 3, n - 1)) * a.stride]);
    }
#pragma unroll
    for (int j = 0; j < NDM; ++j) {
      if (j < nd) {
        const float* sp = S0 + (size_t)(16 * j + 4 * g) * a.e + col;
        const float4 s4 = make_float4(sp[0], sp[a.e], sp[2 * (size_t)a.e], sp[3 * (size_t)a.e]);
#pragma unroll
        for (int tb = 0; tb < 4; ++tb) acc[tb] = lt_mfma4(*(const float4*)&Q_s[16 * tb + r16][16 * j + 4 * g], s4, acc[tb]);
      }
    }
#pragma unroll
    for (int tb = 0; tb < 4; ++tb)
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[tb][i] *= expf(lg * (float)(16 * tb + 4 * g + i + 1));
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const float4 vs = lt_silu4(v[j]);
#pragma unroll
      for (int tb = j; tb < 4; ++tb) acc[tb] = lt_mfma4(*(const float4*)&M_s[16 * tb + r16][16 * j + 4 * g], vs, acc[tb]);
    }
    if (16 * cb + r16 < cols) {
#pragma unroll
      for (int tb = 0; tb < 4; ++tb)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int t = 16 * tb + 4 * g + i;
          if (t < n) a.out[(size_t)(t0 + t) * ((size_t)a.H * a.e) + h * a.e + c0 + col] = acc[tb][i];
        }
    }
  }
}

extern "C" int fg_lightning_chunk_tokens() { return LC; }

// d a multiple of 16 up to 256; columns and stride in multiples of 4, rows 16-byte aligned
extern "C" int fg_lightning_chunk_scan(const LightningArgs* args, const LightningChunks* chunks, int n_chunks, int n_seqs,
                                       hipStream_t stream) {
  if (n_seqs <= 0 || n_chunks <= 0) return FG_OK;
  const LightningArgs& a = *args;
  const LightningChunks& ch = *chunks;
  if (!lightning_ok(a, n_seqs) || n_seqs > 65535 || a.d % 16 || a.d > 256 || a.stride % 4 || a.q_col % 4 || a.k_col % 4 ||
      ((uintptr_t)a.rows & 15) || (long long)a.d * a.e > 2147483647LL || !ch.chunk_start || !ch.seq_chunk || !ch.states)
    return FG_ERR_ARG;
  const dim3 grid(n_chunks, a.H, (a.e + LC_COLS - 1) / LC_COLS);
  const dim3 cgrid((a.d * a.e + 255) / 256, a.H, n_seqs);
#define GO(NDM)                                                              \
  do {                                                                       \
    lightning_chunk_states_kernel<NDM><<<grid, 256, 0, stream>>>(a, ch);     \
    lightning_combine_kernel<<<cgrid, 256, 0, stream>>>(a, ch);              \
    lightning_chunk_out_kernel<NDM><<<grid, 256, 0, stream>>>(a, ch);        \
  } while (0)
  if (a.d <= 64) GO(4);
  else if (a.d <= 128) GO(8);
  else GO(16);
#undef GO
  return fg_launch_status();
}
