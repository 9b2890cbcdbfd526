// Causal softmax attention over the paged cache whose heads' weights are mixed after the softmax, general form: any
// element type, every head of a token in one workgroup.
//
// For query token i (position p) and every key j in its window, per query head h (kv head h / (H / G)):
//   s_h = (q_h . k_j) * scale, then cap * tanh(s_h / cap) if there is a cap
//   p_h = softmax over the visible keys of s_h
//   w_h = sum_g talk[h][g] p_g
//   o_h = sum_j w_h(j) v_j of h's own kv head;   out[i, h, :] = o_h * out_scale
// Mixing needs every head's finished weight of a (query, key) pair, so a workgroup owns a token with all its heads
// and walks the keys twice in tiles of 64 that start at multiples of 64: first every head's maximum and sum (a wave a
// head in turns, a lane a key), then scores again, weights, mixing (a thread a (head, key)), and the product with the
// values (a thread a (head, value dim)).  All arithmetic is fp32, summed in an order that depends on the token's own
// keys alone: not on the batch, the cut of the prompt, or the pages.
//
// Keys and values lie in pages of head size hd_c (kv_layout.h); a key's first d and a value's first e dimensions are
// read.
#include "common.h"
#include "kv_layout.h"

#define MA_THREADS 256
#define MA_WAVES 4
#define MA_TILE 64
#define MA_MAX_ITEMS 16  // (head, value dim) pairs a thread owns at a time: heads * e <= 4096 a pass over the values

struct MixedAttentionArgs {
  const void* q; int q_stride, q_hs;  // q[t, h, :] at t * q_stride + h * q_hs
  const void* k_pages; const void* v_pages;
  const int* block_table; int bt_stride;
  const int* seq_of_token; const int* positions;
  int n_tokens, n_heads, n_kv, d, e, hd_c, page_size;
  float scale, softcap;                // softcap 0: none
  int window;                          // first_key's span
  const float* talk;                   // [n_heads, n_heads]
  float out_scale;
  void* out; int out_stride;           // out[t, h * e + x]
};

template <class T>
__global__ __launch_bounds__(MA_THREADS) void mixed_attention_kernel(const MixedAttentionArgs a) {
  extern __shared__ float lds[];
  const int H = a.n_heads, d8 = (a.d + 7) & ~7;
  float* q_s = lds;                     // [H][d8]
  float* p_s = q_s + H * d8;            // [H][64]: weights
  float* w_s = p_s + H * MA_TILE;       // [H][64]: mixed weights
  float* ml_s = w_s + H * MA_TILE;      // [H][2]: maximum, 1 / sum
  const int tid = threadIdx.x, lane = tid % FG_WAVE, wave = tid / FG_WAVE;
  const int t = blockIdx.x;
  const int seq = a.seq_of_token[t], pos = a.positions[t];
  const int rep = H / a.n_kv, n_items = H * a.e;
  const int first = first_key(pos, a.window), k_begin = first / MA_TILE * MA_TILE;
  const int* table = a.block_table + (size_t)seq * a.bt_stride;
  const KvLayout lay(a.page_size, a.hd_c);
  const size_t head_elems = (size_t)a.page_size * a.hd_c;
  const T* qrow = (const T*)a.q + (size_t)t * a.q_stride;
  for (int i = tid; i < H * d8; i += MA_THREADS) {
    const int h = i / d8, x = i % d8;
    q_s[i] = x < a.d ? to_f<T>(qrow[(size_t)h * a.q_hs + x]) : 0.f;
  }
  __syncthreads();
  const float inv_cap = a.softcap > 0.f ? 1.f / a.softcap : 0.f;
  auto score = [&](int h, int key) -> float {  // a visible key
    const T* khead = (const T*)a.k_pages + ((size_t)table[key / a.page_size] * a.n_kv + h / rep) * head_elems;
    const int kappa = key % a.page_size;
    const float* qh = q_s + h * d8;
    float acc = 0.f;
    for (int x = 0; x < d8; x += 8) {
      float kv[8];
      load8<T>(khead + lay.k_off(kappa, x), kv);
#pragma unroll
      for (int i = 0; i < 8; ++i) acc = fmaf(qh[x + i], kv[i], acc);  // (beyond d the query is zero and the key padded)
    }
    acc *= a.scale;
    return a.softcap > 0.f ? a.softcap * tanhf(acc * inv_cap) : acc;
  };
  // ---- every head's maximum and sum
  for (int h = wave; h < H; h += MA_WAVES) {
    float m = -INFINITY, l = 0.f;
    for (int kb = k_begin; kb <= pos; kb += MA_TILE) {
      const int key = kb + lane;
      const bool valid = key >= first && key <= pos;
      const float s = valid ? score(h, key) : -INFINITY;
      const float m_new = fmaxf(m, wave_max(s));
      l = l * expf(m - m_new) + wave_sum(valid ? expf(s - m_new) : 0.f);  // (every tile holds a visible key)
      m = m_new;
    }
    if (lane == 0) {
      ml_s[2 * h] = m;
      ml_s[2 * h + 1] = 1.f / l;
    }
  }
  // ---- weights, mixing, values; a pass owns MA_MAX_ITEMS * MA_THREADS (head, value dim) pairs
  for (int item0 = 0; item0 < n_items; item0 += MA_MAX_ITEMS * MA_THREADS) {
    float o[MA_MAX_ITEMS];
#pragma unroll
    for (int n = 0; n < MA_MAX_ITEMS; ++n) o[n] = 0.f;
    for (int kb = k_begin; kb <= pos; kb += MA_TILE) {
      __syncthreads();  // the statistics are there; the tile before is done with p_s and w_s
      const int key = kb + lane;
      const bool valid = key >= first && key <= pos;
      for (int h = wave; h < H; h += MA_WAVES)
        p_s[h * MA_TILE + lane] = valid ? expf(score(h, key) - ml_s[2 * h]) * ml_s[2 * h + 1] : 0.f;
      __syncthreads();
      for (int i = tid; i < H * MA_TILE; i += MA_THREADS) {
        const int h = i / MA_TILE, j = i % MA_TILE;
        float w = 0.f;
        for (int g = 0; g < H; ++g) w = fmaf(a.talk[(size_t)h * H + g], p_s[g * MA_TILE + j], w);
        w_s[i] = w;
      }
      __syncthreads();
#pragma unroll
      for (int n = 0; n < MA_MAX_ITEMS; ++n) {
        const int item = item0 + tid + n * MA_THREADS;
        if (item >= n_items) break;
        const int h = item / a.e, x = item % a.e;
        const float* wh = w_s + h * MA_TILE;
        float acc = o[n];
        for (int qd = 0; qd < MA_TILE / 8; ++qd) {  // one stored chunk of eight key slots at a time
          const int base = lay.permuted ? kb + 32 * (qd / 4) + 4 * (qd % 4) : kb + 8 * qd;  // lowest key of the chunk
          const int stride_hi = lay.permuted ? 12 : 0;  // slots 4..7 are 16 keys on
          if (base > pos || base + 7 + stride_hi < first) continue;
          const T* vhead = (const T*)a.v_pages + ((size_t)table[base / a.page_size] * a.n_kv + h / rep) * head_elems;
          float vv[8];
          load8<T>(vhead + lay.v_chunk_off(lay.v_slot(base % a.page_size) / 8, x), vv);
#pragma unroll
          for (int i = 0; i < 8; ++i) {
            const int kk = base + i + (i >= 4 ? stride_hi : 0);
            // select, not multiply: a slot never written may hold anything
            if (kk >= first && kk <= pos) acc = fmaf(wh[kk - kb], vv[i], acc);
          }
        }
        o[n] = acc;
      }
    }
#pragma unroll
    for (int n = 0; n < MA_MAX_ITEMS; ++n) {
      const int item = item0 + tid + n * MA_THREADS;
      if (item < n_items) ((T*)a.out)[(size_t)t * a.out_stride + item] = from_f<T>(o[n] * a.out_scale);
    }
  }
}

extern "C" int fg_mixed_attention(const MixedAttentionArgs* args, int dtype, hipStream_t stream) {
  const MixedAttentionArgs& a = *args;
  if (a.n_tokens <= 0) return FG_OK;
  if (a.n_heads <= 0 || a.n_kv <= 0 || a.n_heads % a.n_kv || a.d <= 0 || a.d > a.hd_c || a.e <= 0 || a.e > a.hd_c ||
      a.hd_c % 8 || a.page_size <= 0 || a.page_size % 8 || a.softcap < 0.f || !a.q || !a.out || !a.k_pages || !a.v_pages ||
      !a.block_table || !a.seq_of_token || !a.positions || !a.talk)
    return FG_ERR_ARG;
  const size_t lds = sizeof(float) * ((size_t)a.n_heads * (((a.d + 7) & ~7) + 2 * MA_TILE + 2));
  if (lds > 160 * 1024 - 256) return FG_ERR_ARG;
#define GO(T)                                                                                                           \
  do {                                                                                                                  \
    if (hipFuncSetAttribute((const void*)mixed_attention_kernel<T>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != \
        hipSuccess)                                                                                                     \
      return FG_ERR_LAUNCH;                                                                                             \
    mixed_attention_kernel<T><<<a.n_tokens, MA_THREADS, lds, stream>>>(a);                                              \
  } while (0)
  if (dtype == FG_F32) GO(float);
  else if (dtype == FG_BF16) GO(bf16_t);
  else return FG_ERR_ARG;
#undef GO
  return fg_launch_status();
}
