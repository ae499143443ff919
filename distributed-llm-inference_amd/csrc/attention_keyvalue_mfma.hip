// Attention whose values are the front of its keys, on the bfloat16 matrix cores: one cached vector of D components
// per token and kv head is the key, its first V components the value (attention over cached latents with a
// rotated part behind them; attention without a value projection). For portions of prompts and single tokens.
//
// Because a kv head's query heads read the same vectors, the rows of a tile are (token, query head) pairs: as many
// whole tokens of an entry as fit 64 rows (one token, 64 heads at a time, where a group is larger), a wave takes
// 16 of them. The tile's visible keys pass through LDS in blocks of 64 (32 where keys are long), read from memory
// once for all rows and for both products, the next block in flight meanwhile. Single tokens of small groups have
// fewer rows than that: then KW waves take the same 16 rows and every KW-th run of 32 keys (LDS holds KW runs), and
// their states meet at the end. Both products run on
// v_mfma_f32_16x16x32_bf16 in transposed form, S^T = K Q^T and O^T = V^T P^T, so a lane holds scores of ONE
// row: of the keys 4 g + i and 16 + 4 g + i (g = lane / 16, i < 4), which are the eight k of the second product
// as they stand; the keys' dims for its other operand come out of the same LDS rows by the transposing read
// (ds_read_b64_tr_b16: sixteen lanes read four rows of sixteen, each gets a column of four). LDS rows are padded by 16
// bytes: sixteen rows' 16-byte pieces then lie in all 64 banks.
//
// Softmax with exp2 (log2 e in the scale), online, in 32-bit; P is rounded to bfloat16 for the second product
// while the running sum keeps the unrounded values, as in the other matrix-core attention. A window; a sink's score
// per query head (one more term of the denominator).
//
// splits > 1 (single tokens): the blocks of 32 keys go round `splits` workgroups, each leaves its unnormalised
// sum, reference point and denominator; csrc/attention_generic.hip merges them.
#include "common.h"

typedef __bf16 kv_bf8 __attribute__((ext_vector_type(8)));
typedef __bf16 kv_bf4 __attribute__((ext_vector_type(4)));
typedef float kv_f4 __attribute__((ext_vector_type(4)));
typedef unsigned kv_u4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) kv_bf4* kv_lds4;

#define KV_KEYS 32

struct KeyValueArgs {
  const bf16_t* q; int64_t q_stride;
  const bf16_t* pages;                         // [pages][kv_heads][page_size][D]
  bf16_t* out; int64_t out_stride;
  const int* q_start; const int* kv_len; const int* block_tables; int table_stride;
  const int* tile_entry; const int* tile_q0;   // nullptr: every entry is one row
  int q_heads, kv_heads, D, V, page_size, tile_tokens;
  float scale; int window;
  const float* sinks;
  float* parts; int splits;                    // [entries][q_heads][splits][V + 2]
};

// Keys of up to 32 DC components; KW waves share 16 rows and deal the keys; a wave takes KS runs of 32 keys at a time.
template <int DC, int KW, int KS>
__global__ __launch_bounds__(256, DC <= 12 ? 2 : 1) void attention_keyvalue_kernel(KeyValueArgs a) {
  constexpr float LOG2E = 1.4426950408889634f, LN2 = 0.6931471805599453f;
  constexpr int LD = 32 * DC + 8;              // a row in LDS
  constexpr int CN = (4 * DC + 7) / 8;         // 16-byte pieces of a key that a thread brings
  constexpr int RW = 4 / KW, ROWS = 16 * RW, KR = KW * KS, KB = KV_KEYS * KR;
  __shared__ __align__(16) bf16_t kt[2][KB * LD];
  const int tid = threadIdx.x, lane = tid % 64, wave = tid / 64, col = lane & 15, grp = lane >> 4;
  const int rw = wave % RW, kw = wave / RW;
  const int tile = a.splits > 1 ? blockIdx.x / a.splits : gridDim.x - 1 - blockIdx.x;   // (a portion's last tiles see most keys)
  const int split = a.splits > 1 ? blockIdx.x % a.splits : 0;
  const int entry = a.tile_entry != nullptr ? a.tile_entry[tile] : tile;
  const int q0 = a.tile_entry != nullptr ? a.tile_q0[tile] : 0;
  const int kvh = blockIdx.y, group = a.q_heads / a.kv_heads, D = a.D, V = a.V, ps = a.page_size;
  const int tok0 = a.q_start[entry], q_len = a.q_start[entry + 1] - tok0;
  const int first_pos = a.kv_len[entry] - q_len;
  const int tokens = min(a.tile_tokens, q_len - q0), rows = tokens * group;
  const int* table = a.block_tables + (int64_t)entry * a.table_stride;
  const int z_lo = blockIdx.z * ROWS;
  if (tokens <= 0 || z_lo >= rows) return;

  const int row_lo = z_lo + rw * 16;                                 // this wave's rows
  const bool wave_live = row_lo < rows, live = row_lo + col < rows;
  const int mine = min(row_lo + col, rows - 1);
  const int t = mine / group, head = kvh * group + mine % group, pos = first_pos + q0 + t;
  // the tile's and the wave's first and last positions
  const int p_lo = first_pos + q0 + z_lo / group, p_hi = first_pos + q0 + min(z_lo + ROWS - 1, rows - 1) / group;
  const int w_lo = first_pos + q0 + min(row_lo, rows - 1) / group;
  const int w_hi = first_pos + q0 + min(row_lo + 15, rows - 1) / group;

  kv_bf8 qb[DC];
  {
    const bf16_t* qr = a.q + (int64_t)(tok0 + q0 + t) * a.q_stride + (int64_t)head * D;
#pragma unroll
    for (int d = 0; d < DC; ++d) {
      const int at = 32 * d + 8 * grp;
      qb[d] = at < D ? *reinterpret_cast<const kv_bf8*>(qr + at) : kv_bf8{};
    }
  }
  const float scale2 = a.scale * LOG2E;
  const float not_seen = scale2 >= 0.f ? -INFINITY : INFINITY;       // times the scale: minus infinity
  kv_f4 acc[2 * DC];
#pragma unroll
  for (int v = 0; v < 2 * DC; ++v) acc[v] = kv_f4{0.f, 0.f, 0.f, 0.f};
  const bool sink = a.sinks != nullptr && split == 0 && kw == 0;     // (counted once)
  float m_run = sink ? a.sinks[head] * LOG2E : -INFINITY;
  float l_run = sink && grp == 0 ? 1.f : 0.f;                        // (sums are lane by lane until the end)

  const int j_first = a.window > 0 ? max(0, p_lo - a.window + 1) : 0;
  const int b_end = p_hi >= 0 ? p_hi / KB + 1 : 0;                   // (a padding row has no keys)
  const int step = max(a.splits, 1);
  // this thread's keys of a block (k_row + 32 n) and its first 16-byte piece of each
  const int k_row = tid >> 3, k_piece = tid & 7, pieces = D / 8;
  int page_next[KR];
  auto look = [&](int b) {                                           // (released or absent pages: any page will do)
#pragma unroll
    for (int n = 0; n < KR; ++n) page_next[n] = max(table[min((b * KB + k_row + 32 * n) / ps, a.table_stride - 1)], 0);
  };
  kv_u4 raw[KR][CN];
  auto fetch = [&](int b) {
#pragma unroll
    for (int n = 0; n < KR; ++n) {
      const bf16_t* kr = a.pages + (((int64_t)page_next[n] * a.kv_heads + kvh) * ps + (b * KB + k_row + 32 * n) % ps) * D;
#pragma unroll
      for (int c = 0; c < CN; ++c) {
        const int piece = k_piece + 8 * c;
        raw[n][c] = *reinterpret_cast<const kv_u4*>(kr + 8 * min(piece, pieces - 1));
        if (piece >= pieces) raw[n][c] = kv_u4{0, 0, 0, 0};
      }
    }
  };
  auto put = [&](int buf) {
#pragma unroll
    for (int n = 0; n < KR; ++n)
#pragma unroll
      for (int c = 0; c < CN; ++c) {
        const int piece = k_piece + 8 * c;
        if (piece < 4 * DC) *reinterpret_cast<kv_u4*>(&kt[buf][(k_row + 32 * n) * LD + 8 * piece]) = raw[n][c];
      }
  };
  int b = j_first / KB + split;
  if (b < b_end) {
    look(b);
    fetch(b);
    put(0);
    look(min(b + step, b_end - 1));
  }
  int buf = 0;
  __syncthreads();
  for (; b < b_end; b += step, buf ^= 1) {
    const bool more = b + step < b_end;
    if (more) {
      fetch(b + step);
      look(min(b + 2 * step, b_end - 1));
    }
    constexpr int WK = KV_KEYS * KS;                                 // keys of a wave at a time
    const int j0 = b * KB + WK * kw;
    if (wave_live && j0 <= w_hi && (a.window <= 0 || j0 + WK - 1 > w_lo - a.window)) {
      const bf16_t* kb = kt[buf] + WK * kw * LD;
      kv_f4 s[2 * KS];
#pragma unroll
      for (int sub = 0; sub < 2 * KS; ++sub) s[sub] = kv_f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int d = 0; d < DC; ++d)
#pragma unroll
        for (int sub = 0; sub < 2 * KS; ++sub)
          s[sub] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              *reinterpret_cast<const kv_bf8*>(&kb[(16 * sub + col) * LD + 32 * d + 8 * grp]), qb[d], s[sub], 0, 0, 0);
      // s[sub][i]: key j0 + 16 sub + 4 grp + i against row `col`
      if (j0 + WK - 1 > w_lo || (a.window > 0 && j0 <= w_hi - a.window)) {   // (else every key is seen by every row)
#pragma unroll
        for (int sub = 0; sub < 2 * KS; ++sub)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int j = j0 + 16 * sub + 4 * grp + i;
            s[sub][i] = j <= pos && (a.window <= 0 || j > pos - a.window) ? s[sub][i] : not_seen;
          }
      }
      // (the largest score is the largest product for a positive scale, the smallest for a negative one)
      float mx = not_seen;
#pragma unroll
      for (int sub = 0; sub < 2 * KS; ++sub)
#pragma unroll
        for (int i = 0; i < 4; ++i) mx = scale2 >= 0.f ? fmaxf(mx, s[sub][i]) : fminf(mx, s[sub][i]);
      mx *= scale2;
      mx = fmaxf(mx, __shfl_xor(mx, 16, DLI_WAVE));
      mx = fmaxf(mx, __shfl_xor(mx, 32, DLI_WAVE));
      const float m_new = fmaxf(m_run, mx);
      const float m_safe = m_new > -INFINITY ? m_new : 0.f;            // (nothing seen yet: every weight is exp2(-inf))
      const float alpha = __builtin_amdgcn_exp2f(m_run - m_safe);
      const bool moved = __any(m_new > m_run);
      float sum = 0.f;
      kv_bf8 pb[KS];
#pragma unroll
      for (int sub = 0; sub < 2 * KS; ++sub)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float p = __builtin_amdgcn_exp2f(fmaf(s[sub][i], scale2, -m_safe));
          sum += p;
          pb[sub / 2][4 * (sub % 2) + i] = (bf16_t)p;
        }
      l_run = l_run * alpha + sum;
      m_run = m_new;
      if (moved) {
#pragma unroll
        for (int v = 0; v < 2 * DC; ++v) acc[v] *= alpha;
      }
      const bf16_t* vb = kb + (4 * grp + col / 4) * LD + 4 * (col % 4);
#pragma unroll
      for (int v = 0; v < 2 * DC; ++v)
        if (16 * v < V) {
#pragma unroll
          for (int k = 0; k < KS; ++k) {
            const bf16_t* vk = vb + KV_KEYS * k * LD + 16 * v;
            const kv_bf4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((kv_lds4)(vk));
            const kv_bf4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((kv_lds4)(vk + 16 * LD));
            const kv_bf8 v8 = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
            acc[v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v8, pb[k], acc[v], 0, 0, 0);
          }
        }
    }
    if (more) put(buf ^ 1);
    __syncthreads();
  }
  if constexpr (KW > 1) {
    // the waves that share rows meet: the others leave their states in LDS (the keys are done with), the first
    // adds them in their order
    constexpr int STATE = (2 * DC * 4 + 2) * 64;                     // floats a wave
    static_assert((KW - 1) * RW * STATE * 4 <= (int)sizeof(kt), "the states fit where the keys were");
    float* mem = reinterpret_cast<float*>(&kt[0][0]);
    if (kw > 0) {
      float* st = mem + ((kw - 1) * RW + rw) * STATE + lane;
#pragma unroll
      for (int v = 0; v < 2 * DC; ++v)
#pragma unroll
        for (int i = 0; i < 4; ++i) st[(4 * v + i) * 64] = acc[v][i];
      st[8 * DC * 64] = m_run;
      st[(8 * DC + 1) * 64] = l_run;
    }
    __syncthreads();
    if (kw > 0) return;
#pragma unroll
    for (int k = 1; k < KW; ++k) {
      const float* st = mem + ((k - 1) * RW + rw) * STATE + lane;
      const float mk = st[8 * DC * 64], m_new = fmaxf(m_run, mk);
      if (m_new > -INFINITY) {
        const float f0 = __builtin_amdgcn_exp2f(m_run - m_new), f1 = __builtin_amdgcn_exp2f(mk - m_new);
#pragma unroll
        for (int v = 0; v < 2 * DC; ++v)
#pragma unroll
          for (int i = 0; i < 4; ++i) acc[v][i] = acc[v][i] * f0 + st[(4 * v + i) * 64] * f1;
        l_run = l_run * f0 + st[(8 * DC + 1) * 64] * f1;
        m_run = m_new;
      }
    }
  }
  float l = l_run + __shfl_xor(l_run, 16, DLI_WAVE);
  l += __shfl_xor(l, 32, DLI_WAVE);
  if (!live) return;
  // acc[v][i] is value 16 v + 4 grp + i of this lane's row
  if (a.splits > 1) {
    float* part = a.parts + (((int64_t)entry * a.q_heads + head) * a.splits + split) * (V + 2);
#pragma unroll
    for (int v = 0; v < 2 * DC; ++v)
      if (16 * v + 4 * grp < V)
#pragma unroll
        for (int i = 0; i < 4; ++i) part[16 * v + 4 * grp + i] = acc[v][i];
    if (grp == 0) {
      part[V] = m_run * LN2;
      part[V + 1] = l;
    }
    return;
  }
  const float inv = l > 0.f ? 1.f / l : 0.f;
  bf16_t* o = a.out + (int64_t)(tok0 + q0 + t) * a.out_stride + (int64_t)head * V;
#pragma unroll
  for (int v = 0; v < 2 * DC; ++v)
    if (16 * v + 4 * grp < V) {
      kv_bf4 y;
#pragma unroll
      for (int i = 0; i < 4; ++i) y[i] = (bf16_t)(acc[v][i] * inv);
      *reinterpret_cast<kv_bf4*>(o + 16 * v + 4 * grp) = y;
    }
}

// Blocks of 32 components that a key of head_dim takes, as built.
static int kv_dc(int head_dim) {
  const int dc = (head_dim + 31) / 32;
  return dc <= 6 ? dc : dc <= 8 ? 8 : dc <= 10 ? dc : dc <= 12 ? 12 : dc <= 16 ? 16 : dc <= 18 ? 18 : 20;
}
// Waves that share the rows of a single token: as many as its heads leave free and LDS holds keys for.
static int kv_kw(int dc, int group) { return group <= 16 && dc <= 4 ? 4 : group <= 32 && dc <= 10 ? 2 : 1; }

extern "C" {

// csrc/attention_generic.hip
int dli_attention_scored_merge_bf16(const float* parts, int splits, int entries, int q_heads, int value_dim, void* out,
                                    int64_t out_stride, hipStream_t stream);

int dli_attention_keyvalue_supports(int head_dim, int value_dim) {
  return head_dim >= 8 && head_dim <= 640 && head_dim % 8 == 0 && value_dim >= 8 && value_dim <= head_dim && value_dim % 8 == 0;
}

// Whole tokens of a tile (the host builds its tile list with this).
int dli_attention_keyvalue_tile_tokens(int q_heads, int kv_heads) {
  if (q_heads <= 0 || kv_heads <= 0 || q_heads % kv_heads != 0) return DLI_ERR_ARGUMENT;
  const int group = q_heads / kv_heads;
  return group >= 64 ? 1 : 64 / group;
}

// How many workgroups share an entry's keys in a step of single tokens: as many as bring the launch to two a
// compute unit, 16 at most. It depends on the heads and the number of entries, never on their lengths.
int dli_attention_keyvalue_splits(int q_heads, int kv_heads, int head_dim, int entries) {
  if (q_heads <= 0 || kv_heads <= 0 || q_heads % kv_heads != 0 || entries <= 0 || head_dim <= 0) return 1;
  const int group = q_heads / kv_heads, rows = 64 / kv_kw(kv_dc(head_dim), group);
  const int64_t workgroups = (int64_t)entries * kv_heads * ((group + rows - 1) / rows);
  const int64_t splits = 512 / workgroups;
  return splits < 1 ? 1 : splits > 16 ? 16 : (int)splits;
}

// tile_entry == nullptr: every entry is one row, tiles = entries. splits > 1 (such steps only): parts is float
// [entries * q_heads * splits * (value_dim + 2)] of scratch.
int dli_attention_keyvalue(const void* q, int64_t q_stride, const void* pages, void* out, int64_t out_stride,
                           const int* q_start, const int* kv_len, const int* block_tables, int table_stride,
                           const int* tile_entry, const int* tile_q0, int tiles, int q_heads, int kv_heads, int head_dim,
                           int value_dim, int page_size, float scale, int window, const float* sinks, float* parts, int splits,
                           hipStream_t stream) {
  if (tiles <= 0) return DLI_OK;
  if (!dli_attention_keyvalue_supports(head_dim, value_dim) || q_heads <= 0 || kv_heads <= 0 || q_heads % kv_heads != 0 ||
      kv_heads > 65535 || page_size <= 0 || table_stride <= 0 || window < 0 || q_stride % 8 != 0 || out_stride % 4 != 0 ||
      (tile_entry == nullptr) != (tile_q0 == nullptr) || splits < 1 || splits > 64 ||
      (splits > 1 && (parts == nullptr || tile_entry != nullptr)) || (int64_t)tiles * splits > 0x7fffffff)
    return DLI_ERR_ARGUMENT;
  KeyValueArgs a;
  a.q = (const bf16_t*)q; a.q_stride = q_stride; a.pages = (const bf16_t*)pages; a.out = (bf16_t*)out; a.out_stride = out_stride;
  a.q_start = q_start; a.kv_len = kv_len; a.block_tables = block_tables; a.table_stride = table_stride;
  a.tile_entry = tile_entry; a.tile_q0 = tile_q0; a.q_heads = q_heads; a.kv_heads = kv_heads; a.D = head_dim; a.V = value_dim;
  a.page_size = page_size; a.scale = scale; a.window = window; a.sinks = sinks; a.parts = parts; a.splits = splits;
  const int group = q_heads / kv_heads, dc = kv_dc(head_dim);
  const bool single = tile_entry == nullptr;
  const int kw = single ? kv_kw(dc, group) : 1, rows = 64 / kw;
  a.tile_tokens = single ? 1 : dli_attention_keyvalue_tile_tokens(q_heads, kv_heads);
  const dim3 grid(tiles * splits, kv_heads, (a.tile_tokens * group + rows - 1) / rows);
  if (grid.z > 65535) return DLI_ERR_ARGUMENT;
#define KV_LAUNCH(DC, KW, KS) attention_keyvalue_kernel<DC, KW, KS><<<grid, 256, 0, stream>>>(a)
#define KV_SMALL(DC)                             \
  case DC:                                       \
    if (!single) KV_LAUNCH(DC, 1, 2);         \
    else if (kw == 4) KV_LAUNCH(DC, 4, 1);    \
    else if (kw == 2) KV_LAUNCH(DC, 2, 1);    \
    else KV_LAUNCH(DC, 1, 1);                 \
    break;
#define KV_MIDDLE(DC)                            \
  case DC:                                       \
    if (!single) KV_LAUNCH(DC, 1, 2);         \
    else if (kw == 2) KV_LAUNCH(DC, 2, 1);    \
    else KV_LAUNCH(DC, 1, 1);                 \
    break;
#define KV_LARGE(DC) case DC: KV_LAUNCH(DC, 1, 1); break;
  switch (dc) {
    KV_SMALL(1) KV_SMALL(2) KV_SMALL(3) KV_SMALL(4)
    KV_MIDDLE(5) KV_MIDDLE(6) KV_MIDDLE(8) KV_MIDDLE(9) KV_MIDDLE(10)
    KV_LARGE(12) KV_LARGE(16) KV_LARGE(18) KV_LARGE(20)
    default: return DLI_ERR_ARGUMENT;
  }
#undef KV_LAUNCH
#undef KV_SMALL
#undef KV_MIDDLE
#undef KV_LARGE
  const int status = dli_launch_status();
  if (status != DLI_OK || splits == 1) return status;
  return dli_attention_scored_merge_bf16(parts, splits, tiles, q_heads, value_dim, out, out_stride, stream);
}

}  // extern "C"
