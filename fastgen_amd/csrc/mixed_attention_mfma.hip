// Causal softmax attention whose heads' weights are mixed after the softmax, on the matrix cores in bfloat16
// (gfx950); see mixed_attention.hip for what it computes.  Compiled once per width of a head in the cache:
// -DFG_HD=<multiple of 16, at most 256>.  At most 16 heads, pages of a multiple of 32 keys.
//
// Prompt portions.  An *item* is up to 16 consecutive query tokens of one sequence with all their heads.
//   1. mixed_stats: every (token, head)'s maximum and sum over its keys (the scores alone; a workgroup an item
//      and a key/value head, its waves take the key tiles in turns).
//   2. mixed_tile: a workgroup an item and a chunk of its keys.  Per tile of 32 keys, with LDS between the phases:
//      scores S_g^T = K Q_g^T per head (v_mfma_f32_16x16x32_bf16; a wave owns a few heads) and finished weights
//      exp(s - m) / l; mixing W = T P over the heads per key: the weights enter as two bfloat16 terms (16
//      significant bits), the two terms of 16 heads side by side in the 32 k of one MFMA (a second one takes what
//      rounding T dropped, if anything); values O_h^T += V^T W_h^T, both terms of W.
//      The weights are finished, so chunks of keys simply add (mixed_tile_combine, in order).
// Decoded tokens.  Mixing is linear, so it may follow the product with the values: with A[g, c] = sum_j p_g(j) v_c(j)
// for every head g and every key/value head c, o_h = sum_g T[h, g] A[g, kv(h)].  The rows of an MFMA are the
// (at most 16) heads, which a plain decode kernel leaves mostly empty, so nothing is lost:
//   mixed_decode: a workgroup a token and a chunk of its keys, waves take tiles of 32 keys: scores of all heads (the
//   products of the key heads accumulate into one tile, each with the queries of its own group), a running softmax,
//   A for the key/value heads of the workgroup; mixed_decode_combine merges the chunks and mixes.
// Positions of keys are taken relative to the first tile an item sees, so a window bounds the number of chunks.
#include "common.h"
#include "kv_layout.h"

#ifndef FG_HD
#error "compile with -DFG_HD=<head size>"
#endif
static_assert(FG_HD % 16 == 0 && FG_HD >= 16 && FG_HD <= 256, "head size: multiple of 16 up to 256");

constexpr int HD = FG_HD;
constexpr int NKS = (HD + 31) / 32;  // 32-wide steps over the head dimension (the last may be half)
constexpr int NDB = HD / 16;         // 16-wide blocks of the head dimension
constexpr int KT = 32;               // keys of a tile
constexpr int TQ = 16;               // query tokens of an item
constexpr int HP = 16;               // heads, padded
constexpr int MT_THREADS = 256;
constexpr int P_LD = 20;             // weights[h][key][token] in words (key rows: lane groups in different banks)
constexpr int P_HS = KT * P_LD + 2;  // ... of a head (heads 8 apart start 16 banks apart)
constexpr int W_LD = KT + 4;         // mixed[h][token][key] in words, rows 16-byte aligned
constexpr int CB = HD >= 512 ? 1 : (512 / HD > 8 ? 8 : 512 / HD);  // key/value heads whose sums a decode workgroup holds
constexpr int MD_MAX_CHUNKS = 256;

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));

struct MixedTileArgs {
  const bf16_t* q; int q_stride, q_hs;  // q[t, h, :] at t * q_stride + h * q_hs
  const bf16_t* k_pages; const bf16_t* v_pages;
  const int* block_table; int bt_stride;
  const int* items; int n_items;        // [n_items, 4]: sequence, first flat token, tokens (<= 16), first position
  int n_tokens, n_heads, n_kv, d, e, page_size;
  float scale, softcap;                 // softcap 0: none
  int window;                           // first_key's span
  const float* talk; int talk_low;      // [n_heads, n_heads]; whether rounding it to bfloat16 drops anything
  float out_scale;
  bf16_t* out; int out_stride;          // out[t, h * e + x]
  float* stats;                         // [n_tokens, n_heads, 2]: maximum (base 2), 1 / sum
  float* partial; int n_chunks, chunk_keys;  // tile: [n_chunks, n_tokens, n_heads * e] or null (one chunk)
  float* part_ml;                       // decode: partial [n_chunks, n_items, n_kv, 16, HD], part_ml [n_chunks, n_items, 16, 2]
};

#define LOG2E 1.4426950408889634f

__device__ __forceinline__ bf16x8 zero8() {
  bf16x8 z;
#pragma unroll
  for (int i = 0; i < 8; ++i) z[i] = (__bf16)0.f;
  return z;
}

// zeroes the value slots of keys beyond `hi`; slot s of a chunk is key ka + (s & 3) + 16 * (s >> 2)
__device__ __forceinline__ bf16x8 mask_slots(bf16x8 v, int ka, int hi) {
  u32x4 m;
#pragma unroll
  for (int w = 0; w < 4; ++w) {
    const int k_even = ka + ((2 * w) & 3) + 16 * ((2 * w) >> 2), k_odd = k_even + 1;
    m[w] = (k_even <= hi ? 0x0000ffffu : 0u) | (k_odd <= hi ? 0xffff0000u : 0u);
  }
  return __builtin_bit_cast(bf16x8, __builtin_bit_cast(u32x4, v) & m);
}

// Raw products to scores in base 2: scale, then cap * tanh(./cap) as cap * (1 - 2 / (1 + exp(2 ./cap))).
struct ScoreFn {
  float mul, cap2;  // without a cap: s * mul; with one: cap2 * (1 - 2 / (1 + exp2(s * mul)))
  bool capped;
  __device__ __forceinline__ ScoreFn(const MixedTileArgs& a) {
    capped = a.softcap > 0.f;
    mul = capped ? 2.f * LOG2E * a.scale / a.softcap : a.scale * LOG2E;
    cap2 = a.softcap * LOG2E;
  }
  __device__ __forceinline__ float operator()(float s) const {
    const float x = s * mul;
    return capped ? cap2 - 2.f * cap2 * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(x)) : x;
  }
};

__device__ __forceinline__ float max_over_groups(float v) {
  const auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  v = fmaxf(__uint_as_float(a[0]), __uint_as_float(a[1]));
  const auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  return fmaxf(__uint_as_float(b[0]), __uint_as_float(b[1]));
}

// what the weight w is in LDS: two bfloat16 terms in one word, the rounded weight in the upper half
__device__ __forceinline__ uint32_t two_terms(float w) {
  const __bf16 hi = (__bf16)w;
  const __bf16 lo = (__bf16)(w - (float)hi);
  return ((uint32_t)__builtin_bit_cast(uint16_t, hi) << 16) | (uint32_t)__builtin_bit_cast(uint16_t, lo);
}

__device__ __forceinline__ void load_query(bf16x8 (&qop)[NKS], const bf16_t* qrow, int d, int g, bool ok) {
#pragma unroll
  for (int ks = 0; ks < NKS; ++ks) {
    bf16x8 v = zero8();
#pragma unroll
    for (int x = 0; x < 8; ++x) {
      const int dim = 32 * ks + 8 * g + x;
      if (ok && dim < d) v[x] = __builtin_bit_cast(__bf16, qrow[dim]);
    }
    qop[ks] = v;
  }
}

// ------------------------------------------------------------------ statistics
// grid (n_items, n_kv); HB heads of the group at a time
template <int HB>
__global__ __launch_bounds__(MT_THREADS) void mixed_stats_kernel(const MixedTileArgs a) {
  __shared__ float ml_s[4][HB][TQ][2];
  const int tid = threadIdx.x, lane = tid % FG_WAVE, wave = tid / FG_WAVE;
  const int g = lane >> 4, row = lane & 15;
  const int4 it = *(const int4*)(a.items + 4 * blockIdx.x);
  const int seq = it.x, tok0 = it.y, n_tok = it.z, pos0 = it.w, kvh = blockIdx.y;
  const int pos_last = pos0 + n_tok - 1, rep = a.n_heads / a.n_kv;
  const bool row_valid = row < n_tok;
  const int pos_row = row_valid ? pos0 + row : -1;
  const int first_row = first_key(pos0 + row, a.window);
  const int k_lo = first_key(pos0, a.window) / KT * KT;
  const int* table = a.block_table + (size_t)seq * a.bt_stride;
  const KvLayout lay(a.page_size, HD);
  const size_t head_elems = (size_t)a.page_size * HD;
  const ScoreFn fn(a);
  for (int h0 = 0; h0 < rep; h0 += HB) {
    bf16x8 qop[HB][NKS];
    float m[HB], l[HB];
#pragma unroll
    for (int j = 0; j < HB; ++j) {
      const int h = kvh * rep + min(h0 + j, rep - 1);
      load_query(qop[j], a.q + (size_t)(tok0 + (row_valid ? row : 0)) * a.q_stride + (size_t)h * a.q_hs, a.d, g, row_valid);
      m[j] = -INFINITY;
      l[j] = 0.f;
    }
    bf16x8 kop[2][NKS];
    auto ask = [&](int k0) {  // a tile lies in one page; its first key or a later one is visible, so the page is there
      const bf16_t* kp = a.k_pages + ((size_t)table[k0 / a.page_size] * a.n_kv + kvh) * head_elems;
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int ks = 0; ks < NKS; ++ks) {
          const int dim = 32 * ks + 8 * g;
          kop[kb][ks] = dim < HD ? *(const bf16x8*)(kp + lay.k_off(k0 % a.page_size + 16 * kb + row, dim < HD ? dim : 0)) : zero8();
        }
    };
    int k0 = k_lo + wave * KT;
    if (k0 <= pos_last) ask(k0);
    for (; k0 <= pos_last; k0 += 4 * KT) {
      f32x4 s[2][HB];
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int j = 0; j < HB; ++j) {
          s[kb][j] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int ks = 0; ks < NKS; ++ks)
            s[kb][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kop[kb][ks], qop[j][ks], s[kb][j], 0, 0, 0);
        }
      if (k0 + 4 * KT <= pos_last) ask(k0 + 4 * KT);
#pragma unroll
      for (int j = 0; j < HB; ++j) {
        float v[8], mx = -INFINITY;
#pragma unroll
        for (int kb = 0; kb < 2; ++kb)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int key = k0 + 16 * kb + 4 * g + i;
            const float x = fn(s[kb][j][i]);
            v[4 * kb + i] = ((key >= first_row) & (key <= pos_row)) ? x : -INFINITY;
            mx = fmaxf(mx, v[4 * kb + i]);
          }
        const float m_new = fmaxf(m[j], mx), m_use = m_new == -INFINITY ? 0.f : m_new;  // (this lane's own keys)
        float sum = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) sum += __builtin_amdgcn_exp2f(v[i] - m_use);
        l[j] = l[j] * __builtin_amdgcn_exp2f(m[j] - m_use) + sum;
        m[j] = m_new;
      }
    }
    __syncthreads();  // the heads before are done with ml_s
#pragma unroll
    for (int j = 0; j < HB; ++j) {
      const float M = max_over_groups(m[j]);
      float L = M == -INFINITY ? 0.f : l[j] * __builtin_amdgcn_exp2f(m[j] - M);
      L += __shfl_xor(L, 16, FG_WAVE);
      L += __shfl_xor(L, 32, FG_WAVE);
      if (g == 0) {
        ml_s[wave][j][row][0] = M;
        ml_s[wave][j][row][1] = L;
      }
    }
    __syncthreads();
    for (int i = tid; i < HB * TQ; i += MT_THREADS) {
      const int j = i / TQ, r = i % TQ;
      if (r < n_tok && h0 + j < rep) {
        float M = -INFINITY, L = 0.f;
#pragma unroll
        for (int w = 0; w < 4; ++w) M = fmaxf(M, ml_s[w][j][r][0]);
#pragma unroll
        for (int w = 0; w < 4; ++w)
          L += ml_s[w][j][r][0] == -INFINITY ? 0.f : ml_s[w][j][r][1] * __builtin_amdgcn_exp2f(ml_s[w][j][r][0] - M);
        float* st = a.stats + ((size_t)(tok0 + r) * a.n_heads + kvh * rep + h0 + j) * 2;
        st[0] = M;
        st[1] = 1.f / L;
      }
    }
  }
}

// ------------------------------------------------------------------ prompt portions
// NW waves with HPW heads each.  KV1: the heads of a wave all belong to one kv head; its operands are then kept once and asked for ahead of their use
// (the next tile's keys before the mixing of this one, this tile's values before its scores).
template <int NW, int HPW, bool KV1>
__global__ __launch_bounds__(NW* FG_WAVE) void mixed_tile_kernel(const MixedTileArgs a) {
  extern __shared__ __attribute__((aligned(16))) uint32_t words[];
  uint32_t* wts = words;                                  // [HP][TQ][W_LD]: mixed weights
  uint32_t* prob = words + HP * TQ * W_LD;                // [HP] heads of P_HS: weights
  const int tid = threadIdx.x, lane = tid % FG_WAVE, wave = tid / FG_WAVE;
  const int g = lane >> 4, row = lane & 15;
  const int4 it = *(const int4*)(a.items + 4 * blockIdx.x);
  const int seq = it.x, tok0 = it.y, n_tok = it.z, pos0 = it.w;
  const int pos_last = pos0 + n_tok - 1;
  const int chunk = blockIdx.y;
  const int k_begin = first_key(pos0, a.window) / KT * KT + chunk * a.chunk_keys;
  if (k_begin > pos_last) return;  // uniform
  const int k_last = min(pos_last, k_begin + a.chunk_keys - 1);
  const int H = a.n_heads, rep = H / a.n_kv;
  const bool row_valid = row < n_tok;
  const int pos_row = row_valid ? pos0 + row : -1;
  const int first_row = first_key(pos0 + row, a.window);
  const int* table = a.block_table + (size_t)seq * a.bt_stride;
  const KvLayout lay(a.page_size, HD);
  const size_t head_elems = (size_t)a.page_size * HD;
  const ScoreFn fn(a);

  for (int i = tid; i < HP * P_HS; i += NW * FG_WAVE) prob[i] = 0u;  // the rows of heads that do not exist stay zero

  // this wave's heads: their queries as operands, their statistics, their sums
  bf16x8 qop[HPW][NKS];
  float st_m[HPW], st_l[HPW];
  f32x4 o[HPW][NDB];
#pragma unroll
  for (int j = 0; j < HPW; ++j) {
    const int h = wave * HPW + j;
    const size_t t = (size_t)(tok0 + (row_valid ? row : 0));
    load_query(qop[j], a.q + t * a.q_stride + (size_t)(h < H ? h : 0) * a.q_hs, a.d, g, row_valid && h < H);
    const float2 st = *(const float2*)(a.stats + (t * H + (h < H ? h : 0)) * 2);
    st_m[j] = st.x;
    st_l[j] = st.y;
#pragma unroll
    for (int db = 0; db < NDB; ++db) o[j][db] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  // the mixing matrix as the products' first operand, A[m = lane % 16][k = 8 (lane / 16) + x]: heads 8 (g & 1) + x,
  // for the weights' upper terms (g < 2) and for the lower ones
  bf16x8 talk_hi, talk_lo;
#pragma unroll
  for (int x = 0; x < 8; ++x) {
    const int from = 8 * (g & 1) + x;
    const float v = row < H && from < H ? a.talk[row * H + from] : 0.f;
    talk_hi[x] = (__bf16)v;
    talk_lo[x] = (__bf16)(v - (float)talk_hi[x]);
  }

  const int my_kv = min(wave * HPW, H - 1) / rep;
  bf16x8 kpre[KT / 16][NKS], vpre[NDB];
  auto ask_keys = [&](int k0) {
    const bf16_t* kp = a.k_pages + ((size_t)table[k0 / a.page_size] * a.n_kv + my_kv) * head_elems;
#pragma unroll
    for (int kb = 0; kb < KT / 16; ++kb)
#pragma unroll
      for (int ks = 0; ks < NKS; ++ks) {
        const int dim = 32 * ks + 8 * g;
        kpre[kb][ks] = dim < HD ? *(const bf16x8*)(kp + lay.k_off(k0 % a.page_size + 16 * kb + row, dim < HD ? dim : 0)) : zero8();
      }
  };
  auto ask_values = [&](int k0) {
    const bf16_t* vhead = a.v_pages + ((size_t)table[k0 / a.page_size] * a.n_kv + my_kv) * head_elems;
    const int kc = (k0 % a.page_size) / 8 + g;
#pragma unroll
    for (int db = 0; db < NDB; ++db) vpre[db] = *(const bf16x8*)(vhead + lay.v_chunk_off(kc, 16 * db + row));
  };
  // the weights of one head's 16 keys from kb on, finished, to LDS
  auto put_weights = [&](int h, int j, int k0, int kb, const f32x4& s) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int key = k0 + 16 * kb + 4 * g + i;
      const bool visible = (key >= first_row) & (key <= pos_row);
      const float w = __builtin_amdgcn_exp2f(fn(s[i]) - st_m[j]) * st_l[j];
      prob[h * P_HS + (16 * kb + 4 * g + i) * P_LD + row] = visible ? two_terms(w) : 0u;
    }
  };
  if (KV1) ask_keys(k_begin);

  for (int k0 = k_begin; k0 <= k_last; k0 += KT) {
    __syncthreads();  // prob is zeroed; the tile before is done with prob (its mixed weights are read behind a barrier below)
    // ---- 1. scores and weights
    if (KV1) {
      ask_values(k0);
#pragma unroll
      for (int kb = 0; kb < KT / 16; ++kb)
#pragma unroll
        for (int j = 0; j < HPW; ++j) {
          const int h = wave * HPW + j;
          if (h < H) {  // uniform in the wave
            f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < NKS; ++ks) s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kpre[kb][ks], qop[j][ks], s, 0, 0, 0);
            put_weights(h, j, k0, kb, s);
          }
        }
      if (k0 + KT <= k_last) ask_keys(k0 + KT);
    } else {
      const bf16_t* kpage = a.k_pages + (size_t)table[k0 / a.page_size] * a.n_kv * head_elems;
#pragma unroll
      for (int kb = 0; kb < KT / 16; ++kb) {
        bf16x8 kop[NKS];
        int loaded = -1;
#pragma unroll
        for (int j = 0; j < HPW; ++j) {
          const int h = wave * HPW + j;
          if (h < H) {
            const int kvh = h / rep;
            if (kvh != loaded) {  // uniform in the wave
              loaded = kvh;
#pragma unroll
              for (int ks = 0; ks < NKS; ++ks) {
                const int dim = 32 * ks + 8 * g;
                kop[ks] = dim < HD ? *(const bf16x8*)(kpage + (size_t)kvh * head_elems +
                                                      lay.k_off(k0 % a.page_size + 16 * kb + row, dim < HD ? dim : 0)) : zero8();
              }
            }
            f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < NKS; ++ks) s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kop[ks], qop[j][ks], s, 0, 0, 0);
            put_weights(h, j, k0, kb, s);
          }
        }
      }
    }
    __syncthreads();
    // ---- 2. mixing: four keys of a wave at a time; a lane ends with 4 heads of (token, four keys)
#pragma unroll
    for (int kq = 0; kq < KT / (4 * NW); ++kq) {
      const int k4 = (KT / NW) * wave + 4 * kq;
      f32x4 mixed[4];
#pragma unroll
      for (int kk = 0; kk < 4; ++kk) {
        uint32_t p[8];
#pragma unroll
        for (int x = 0; x < 8; ++x) p[x] = prob[(8 * (g & 1) + x) * P_HS + (k4 + kk) * P_LD + row];
        u32x4 packed;
#pragma unroll
        for (int w = 0; w < 4; ++w)
          packed[w] = g < 2 ? (p[2 * w] >> 16) | (p[2 * w + 1] & 0xffff0000u) : (p[2 * w] & 0xffffu) | (p[2 * w + 1] << 16);
        const bf16x8 pop = __builtin_bit_cast(bf16x8, packed);
        f32x4 m = __builtin_amdgcn_mfma_f32_16x16x32_bf16(talk_hi, pop, f32x4{0.f, 0.f, 0.f, 0.f}, 0, 0, 0);
        if (a.talk_low) m = __builtin_amdgcn_mfma_f32_16x16x32_bf16(talk_lo, pop, m, 0, 0, 0);  // uniform
        mixed[kk] = m;
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const u32x4 w4 = {two_terms(mixed[0][i]), two_terms(mixed[1][i]), two_terms(mixed[2][i]), two_terms(mixed[3][i])};
        *(u32x4*)(wts + ((4 * g + i) * TQ + row) * W_LD + k4) = w4;
      }
    }
    __syncthreads();
    // ---- 3. values (a kv head's operands are read once for the heads of its group that follow each other)
    const int page = table[k0 / a.page_size];
    const int kc = (k0 % a.page_size) / 8 + g;
    bf16x8 vop[NDB];
    int loaded = -1;
    if (KV1) {
      loaded = my_kv;
#pragma unroll
      for (int db = 0; db < NDB; ++db) vop[db] = mask_slots(vpre[db], k0 + 4 * g, pos_last);
    }
#pragma unroll
    for (int j = 0; j < HPW; ++j) {
      const int h = wave * HPW + j;
      if (h < H) {
        const int kvh = h / rep;
        if (kvh != loaded) {
          loaded = kvh;
          const bf16_t* vhead = a.v_pages + ((size_t)page * a.n_kv + kvh) * head_elems;
#pragma unroll
          for (int db = 0; db < NDB; ++db)  // a slot never written may hold anything: masked
            vop[db] = mask_slots(*(const bf16x8*)(vhead + lay.v_chunk_off(kc, 16 * db + row)), k0 + 4 * g, pos_last);
        }
        const uint32_t* wr = wts + (h * TQ + row) * W_LD;
        const u32x4 w0 = *(const u32x4*)(wr + 4 * g), w1 = *(const u32x4*)(wr + 16 + 4 * g);
        u32x4 hi, lo;  // eight bfloat16 each: keys 4g..4g+3 and 16+4g..16+4g+3
#pragma unroll
        for (int w = 0; w < 2; ++w) {
          hi[w] = (w0[2 * w] >> 16) | (w0[2 * w + 1] & 0xffff0000u);
          hi[2 + w] = (w1[2 * w] >> 16) | (w1[2 * w + 1] & 0xffff0000u);
          lo[w] = (w0[2 * w] & 0xffffu) | (w0[2 * w + 1] << 16);
          lo[2 + w] = (w1[2 * w] & 0xffffu) | (w1[2 * w + 1] << 16);
        }
        const bf16x8 p_hi = __builtin_bit_cast(bf16x8, hi), p_lo = __builtin_bit_cast(bf16x8, lo);
#pragma unroll
        for (int db = 0; db < NDB; ++db) {
          o[j][db] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vop[db], p_hi, o[j][db], 0, 0, 0);
          o[j][db] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vop[db], p_lo, o[j][db], 0, 0, 0);
        }
      }
    }
  }
  // ---- this lane's sums: token `row`, dimensions 16 db + 4 g + i of its wave's heads
  if (!row_valid) return;
  const int t = tok0 + row, n_cols = H * a.e;
#pragma unroll
  for (int j = 0; j < HPW; ++j) {
    const int h = wave * HPW + j;
    if (h >= H) continue;
#pragma unroll
    for (int db = 0; db < NDB; ++db)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int dim = 16 * db + 4 * g + i;
        if (dim < a.e) {
          if (a.partial) a.partial[((size_t)chunk * a.n_tokens + t) * n_cols + h * a.e + dim] = o[j][db][i];
          else a.out[(size_t)t * a.out_stride + h * a.e + dim] = from_f<bf16_t>(o[j][db][i] * a.out_scale);
        }
      }
  }
}

// out[t, x] = (sum over its item's chunks, in order) * out_scale; grid (items, 16 tokens, columns / 256)
__global__ __launch_bounds__(MT_THREADS) void mixed_tile_combine_kernel(const MixedTileArgs a) {
  const int4 it = *(const int4*)(a.items + 4 * blockIdx.x);
  if ((int)blockIdx.y >= it.z) return;
  const int t = it.y + blockIdx.y, n_cols = a.n_heads * a.e;
  const int x = blockIdx.z * MT_THREADS + threadIdx.x;
  if (x >= n_cols) return;
  const int k_lo = first_key(it.w, a.window) / KT * KT;
  const int n_chunks = (it.w + it.z - 1 - k_lo) / a.chunk_keys + 1;
  const size_t step = (size_t)a.n_tokens * n_cols;
  const float* p = a.partial + (size_t)t * n_cols + x;
  float y = 0.f;
  int c = 0;
  for (; c + 4 <= n_chunks; c += 4) {  // four loads in flight, added in order
    const float p0 = p[c * step], p1 = p[(c + 1) * step], p2 = p[(c + 2) * step], p3 = p[(c + 3) * step];
    y += p0; y += p1; y += p2; y += p3;
  }
  for (; c < n_chunks; ++c) y += p[c * step];
  a.out[(size_t)t * a.out_stride + x] = from_f<bf16_t>(y * a.out_scale);
}

// ------------------------------------------------------------------ decoded tokens
// grid (n_items, n_chunks, ceil(n_kv / CB)); an item is one token
__global__ __launch_bounds__(MT_THREADS) void mixed_decode_kernel(const MixedTileArgs a) {
  extern __shared__ __attribute__((aligned(16))) char lds[];
  bf16x8* q_s = (bf16x8*)lds;  // [n_kv][NKS][64 lanes]: the queries of each group
  float* o_s = (float*)lds;  // in their place once the waves have ended their keys: [2][CB][NDB][64 lanes][4]
  __shared__ float ml_s[2][HP][2];
  const int tid = threadIdx.x, lane = tid % FG_WAVE, wave = tid / FG_WAVE;
  const int g = lane >> 4, row = lane & 15;
  const int4 it = *(const int4*)(a.items + 4 * blockIdx.x);
  const int seq = it.x, t = it.y, pos = it.w;
  const int chunk = blockIdx.y, c0 = blockIdx.z * CB;
  const int first = first_key(pos, a.window);
  const int k_begin = first / KT * KT + chunk * a.chunk_keys;
  if (k_begin > pos) return;  // uniform
  const int k_last = min(pos, k_begin + a.chunk_keys - 1);
  const int H = a.n_heads, G = a.n_kv, rep = H / G;
  const int* table = a.block_table + (size_t)seq * a.bt_stride;
  const KvLayout lay(a.page_size, HD);
  const size_t head_elems = (size_t)a.page_size * HD;
  const ScoreFn fn(a);
  for (int i = wave; i < G * NKS; i += MT_THREADS / FG_WAVE) {
    const int c = i / NKS, ks = i % NKS;
    bf16x8 v = zero8();
    if (row < H && row / rep == c) {
      const bf16_t* qrow = a.q + (size_t)t * a.q_stride + (size_t)row * a.q_hs;
#pragma unroll
      for (int x = 0; x < 8; ++x) {
        const int dim = 32 * ks + 8 * g + x;
        if (dim < a.d) v[x] = __builtin_bit_cast(__bf16, qrow[dim]);
      }
    }
    q_s[i * FG_WAVE + lane] = v;
  }
  __syncthreads();

  float m = -INFINITY, l = 0.f;
  f32x4 o[CB][NDB];
#pragma unroll
  for (int c = 0; c < CB; ++c)
#pragma unroll
    for (int db = 0; db < NDB; ++db) o[c][db] = f32x4{0.f, 0.f, 0.f, 0.f};

  for (int k0 = k_begin + wave * KT; k0 <= k_last; k0 += 4 * KT) {
    const size_t page = (size_t)table[k0 / a.page_size] * G;
    const int kin = k0 % a.page_size;
    f32x4 s[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
    for (int c = 0; c < G; ++c) {
      const bf16_t* kp = a.k_pages + (page + c) * head_elems;
      bf16x8 kop[2][NKS];
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int ks = 0; ks < NKS; ++ks) {
          const int dim = 32 * ks + 8 * g;
          const bf16x8 v = *(const bf16x8*)(kp + lay.k_off(kin + 16 * kb + row, dim < HD ? dim : 0));
          kop[kb][ks] = dim < HD ? v : zero8();
        }
#pragma unroll
      for (int ks = 0; ks < NKS; ++ks) {
        const bf16x8 qv = q_s[(c * NKS + ks) * FG_WAVE + lane];
#pragma unroll
        for (int kb = 0; kb < 2; ++kb) s[kb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kop[kb][ks], qv, s[kb], 0, 0, 0);
      }
    }
    float v[8], mx = -INFINITY;
#pragma unroll
    for (int kb = 0; kb < 2; ++kb)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int key = k0 + 16 * kb + 4 * g + i;
        const float x = fn(s[kb][i]);
        v[4 * kb + i] = ((key >= first) & (key <= pos)) ? x : -INFINITY;  // (whatever an unwritten key gave)
        mx = fmaxf(mx, v[4 * kb + i]);
      }
    mx = max_over_groups(mx);
    const float m_new = fmaxf(m, mx), m_use = m_new == -INFINITY ? 0.f : m_new;
    const float alpha = __builtin_amdgcn_exp2f(m - m_use);
    float sum = 0.f;
    bf16x8 p_hi, p_lo;  // slots of a value chunk: keys 4g..4g+3 and 16+4g..16+4g+3
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const float p = __builtin_amdgcn_exp2f(v[i] - m_use);
      sum += p;
      p_hi[i] = (__bf16)p;
      p_lo[i] = (__bf16)(p - (float)p_hi[i]);
    }
    l = l * alpha + sum;
    if (__builtin_amdgcn_ballot_w64(m_new != m) != 0) {
#pragma unroll
      for (int c = 0; c < CB; ++c)
#pragma unroll
        for (int db = 0; db < NDB; ++db) o[c][db] *= alpha;
    }
    m = m_new;
    const int kc = kin / 8 + g;
#pragma unroll
    for (int c = 0; c < CB; ++c) {
      if (c0 + c < G) {  // uniform
        const bf16_t* vhead = a.v_pages + (page + c0 + c) * head_elems;
        bf16x8 vop[NDB];
#pragma unroll
        for (int db = 0; db < NDB; ++db) vop[db] = *(const bf16x8*)(vhead + lay.v_chunk_off(kc, 16 * db + row));
#pragma unroll
        for (int db = 0; db < NDB; ++db) {
          const bf16x8 vm = mask_slots(vop[db], k0 + 4 * g, pos);
          o[c][db] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vm, p_hi, o[c][db], 0, 0, 0);
          o[c][db] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vm, p_lo, o[c][db], 0, 0, 0);
        }
      }
    }
  }
  l += __shfl_xor(l, 16, FG_WAVE);
  l += __shfl_xor(l, 32, FG_WAVE);
  // ---- merge the 4 waves pairwise: 2, 3 -> 0, 1, then 1 -> 0; all waves hold the same rows in the same lanes
  auto put = [&](int slot) {
    if (g == 0) {
      ml_s[slot][row][0] = m;
      ml_s[slot][row][1] = l;
    }
#pragma unroll
    for (int c = 0; c < CB; ++c)
#pragma unroll
      for (int db = 0; db < NDB; ++db) *(f32x4*)(o_s + ((((size_t)slot * CB + c) * NDB + db) * FG_WAVE + lane) * 4) = o[c][db];
  };
  auto take = [&](int slot) {
    const float mo = ml_s[slot][row][0], lo = ml_s[slot][row][1];
    const float M = fmaxf(m, mo);
    const float fs = m == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m - M);
    const float fo = mo == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(mo - M);
    l = fs * l + fo * lo;
    m = M;
#pragma unroll
    for (int c = 0; c < CB; ++c)
#pragma unroll
      for (int db = 0; db < NDB; ++db) {
        const f32x4 other = *(const f32x4*)(o_s + ((((size_t)slot * CB + c) * NDB + db) * FG_WAVE + lane) * 4);
        o[c][db] = fs * o[c][db] + fo * other;
      }
  };
  __syncthreads();  // (the queries are no longer read)
  if (wave >= 2) put(wave - 2);
  __syncthreads();
  if (wave < 2) take(wave);
  __syncthreads();
  if (wave == 1) put(0);
  __syncthreads();
  if (wave != 0) return;
  take(0);
  const size_t ci = (size_t)chunk * a.n_items + blockIdx.x;
#pragma unroll
  for (int c = 0; c < CB; ++c) {
    if (c0 + c < G) {
      float* po = a.partial + ((ci * G + c0 + c) * HP + row) * HD;
#pragma unroll
      for (int db = 0; db < NDB; ++db) *(f32x4*)(po + 16 * db + 4 * g) = o[c][db];
    }
  }
  if (g == 0 && c0 == 0) {
    a.part_ml[(ci * HP + row) * 2] = m;
    a.part_ml[(ci * HP + row) * 2 + 1] = l;
  }
}

// grid (n_items, n_kv, ceil(e / 64)); merges the chunks of an item for 64 value dims of one kv head and mixes the heads
__global__ __launch_bounds__(MT_THREADS) void mixed_decode_combine_kernel(const MixedTileArgs a) {
  __shared__ float f_s[HP][MD_MAX_CHUNKS];  // weight of each chunk's sums: 2^(m - M) / L
  __shared__ float a_s[HP][64];
  const int tid = threadIdx.x, lane = tid % FG_WAVE, wave = tid / FG_WAVE;
  const int4 it = *(const int4*)(a.items + 4 * blockIdx.x);
  const int t = it.y, pos = it.w, c = blockIdx.y;
  const int H = a.n_heads, G = a.n_kv, rep = H / G;
  const int k_lo = first_key(pos, a.window) / KT * KT;
  const int n_chunks = (pos - k_lo) / a.chunk_keys + 1;
  for (int r = wave; r < H; r += 4) {
    float M = -INFINITY, L = 0.f;
    for (int s = lane; s < n_chunks; s += FG_WAVE) M = fmaxf(M, a.part_ml[(((size_t)s * a.n_items + blockIdx.x) * HP + r) * 2]);
    M = wave_max(M);
    for (int s = lane; s < n_chunks; s += FG_WAVE) {
      const float2 ml = *(const float2*)(a.part_ml + (((size_t)s * a.n_items + blockIdx.x) * HP + r) * 2);
      const float f = ml.x == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(ml.x - M);
      f_s[r][s] = f;
      L += f * ml.y;
    }
    L = wave_sum(L);
    const float inv = 1.f / L;
    for (int s = lane; s < n_chunks; s += FG_WAVE) f_s[r][s] *= inv;
  }
  __syncthreads();
  const int x = blockIdx.z * 64 + lane;
  const bool x_ok = x < a.e;
  for (int r = wave; r < H; r += 4) {
    float y = 0.f;
    const size_t step = (size_t)a.n_items * G * HP * HD;
    const float* p = a.partial + (((size_t)blockIdx.x * G + c) * HP + r) * HD + min(x, a.e - 1);
    for (int s = 0; s < n_chunks; s += 4) {
      float v[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) v[u] = p[(size_t)min(s + u, n_chunks - 1) * step];
#pragma unroll
      for (int u = 0; u < 4; ++u) y += s + u < n_chunks ? f_s[r][s + u] * v[u] : 0.f;
    }
    a_s[r][lane] = y;
  }
  __syncthreads();
  for (int j = wave; j < rep; j += 4) {
    const int h = c * rep + j;
    float y = 0.f;
    for (int r = 0; r < H; ++r) y = fmaf(a.talk[h * H + r], a_s[r][lane], y);
    if (x_ok) a.out[(size_t)t * a.out_stride + h * a.e + x] = from_f<bf16_t>(y * a.out_scale);
  }
}

static bool mixed_ok(const MixedTileArgs& a) {
  return a.n_heads > 0 && a.n_heads <= HP && a.n_kv > 0 && a.n_heads % a.n_kv == 0 && a.d > 0 && a.d <= HD && a.e > 0 &&
         a.e <= HD && a.page_size > 0 && a.page_size % 32 == 0 && a.softcap >= 0.f && a.chunk_keys >= KT &&
         a.chunk_keys % KT == 0 && a.n_chunks >= 1 && a.n_chunks <= 65535 && a.q && a.out && a.k_pages && a.v_pages &&
         a.block_table && a.items && a.talk && !((uintptr_t)a.items & 15) && a.out_stride >= a.n_heads * a.e;
}

// items of up to 16 tokens; every item's key range has at most n_chunks chunks
extern "C" int fg_mixed_attention_tiles(const MixedTileArgs* args, hipStream_t stream) {
  const MixedTileArgs& a = *args;
  if (a.n_items <= 0) return FG_OK;
  if (!mixed_ok(a) || !a.stats || (a.n_chunks > 1 && !a.partial)) return FG_ERR_ARG;
  const int rep = a.n_heads / a.n_kv;
  const dim3 sgrid(a.n_items, a.n_kv);
  if (rep == 1) mixed_stats_kernel<1><<<sgrid, MT_THREADS, 0, stream>>>(a);
  else if (rep == 2) mixed_stats_kernel<2><<<sgrid, MT_THREADS, 0, stream>>>(a);
  else if (rep == 3) mixed_stats_kernel<3><<<sgrid, MT_THREADS, 0, stream>>>(a);
  else mixed_stats_kernel<4><<<sgrid, MT_THREADS, 0, stream>>>(a);
  const size_t lds = ((size_t)HP * TQ * W_LD + (size_t)HP * P_HS) * sizeof(uint32_t);
  const dim3 grid(a.n_items, a.n_chunks);
#define GO(NW, HPW, KV1)                                                                                                 \
  do {                                                                                                                   \
    if (hipFuncSetAttribute((const void*)mixed_tile_kernel<NW, HPW, KV1>, hipFuncAttributeMaxDynamicSharedMemorySize,    \
                            (int)lds) != hipSuccess)                                                                     \
      return FG_ERR_LAUNCH;                                                                                              \
    mixed_tile_kernel<NW, HPW, KV1><<<grid, NW * FG_WAVE, lds, stream>>>(a);                                             \
  } while (0)
  constexpr bool AHEAD = HD <= 160;  // (wider heads: the operands in flight would not fit the registers)
  if (a.n_heads <= 4) GO(4, 1, true);
  else if (a.n_heads <= 8) GO(8, 1, AHEAD);
  else if (rep % 2 == 0) GO(8, 2, AHEAD);
  else GO(8, 2, false);
#undef GO
  if (a.partial)
    mixed_tile_combine_kernel<<<dim3(a.n_items, TQ, (a.n_heads * a.e + MT_THREADS - 1) / MT_THREADS), MT_THREADS, 0, stream>>>(a);
  return fg_launch_status();
}

extern "C" int fg_mixed_attention_max_chunks() { return MD_MAX_CHUNKS; }

// items of one token
extern "C" int fg_mixed_attention_decode(const MixedTileArgs* args, hipStream_t stream) {
  const MixedTileArgs& a = *args;
  if (a.n_items <= 0) return FG_OK;
  if (!mixed_ok(a) || !a.partial || !a.part_ml || a.n_chunks > MD_MAX_CHUNKS) return FG_ERR_ARG;
  const int q_units = a.n_kv * NKS, o_units = 2 * CB * NDB;  // at most 128 and 64: n_kv <= 16, HD <= 256
  const size_t lds = (size_t)(q_units > o_units ? q_units : o_units) * FG_WAVE * 16;
  if (hipFuncSetAttribute((const void*)mixed_decode_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)
    return FG_ERR_LAUNCH;
  mixed_decode_kernel<<<dim3(a.n_items, a.n_chunks, (a.n_kv + CB - 1) / CB), MT_THREADS, lds, stream>>>(a);
  mixed_decode_combine_kernel<<<dim3(a.n_items, a.n_kv, (a.e + 63) / 64), MT_THREADS, 0, stream>>>(a);
  return fg_launch_status();
}
