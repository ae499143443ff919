// Attention whose values are the front of its keys, on the bfloat16 matrix cores: one cached vector of D components
// per token and kv head is the key, its first V components the value (attention over cached latents with a
// rotated part behind them; attention without a value projection). For portions of prompts and single tokens.
//
// Because a kv head's query heads read the same vectors, the rows of a tile are (token, query head) pairs: 64
// rows are as many whole tokens of an entry as fit (one token, 64 heads at a time, where a group is larger), a
// wave takes 16 of them. The tile's visible keys pass through LDS 32 at a time, read from memory once for all
// rows and for both products, the next 32 in flight meanwhile. Both products run on
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

#define KV_ROWS 64
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

template <int DC>   // keys of up to 32 DC components
__global__ __launch_bounds__(256, DC <= 12 ? 2 : 1) void attention_keyvalue_kernel(KeyValueArgs a) {
  constexpr float LOG2E = 1.4426950408889634f, LN2 = 0.6931471805599453f;
  constexpr int LD = 32 * DC + 8;              // a row in LDS
  constexpr int CN = (4 * DC + 7) / 8;         // 16-byte pieces of a key that a thread brings
  __shared__ __align__(16) bf16_t kt[2][KV_KEYS * LD];
  const int tid = threadIdx.x, lane = tid % 64, wave = tid / 64, col = lane & 15, grp = lane >> 4;
  const int tile = a.splits > 1 ? blockIdx.x / a.splits : gridDim.x - 1 - blockIdx.x;   // (a portion's last tiles see most keys)
  const int split = a.splits > 1 ? blockIdx.x % a.splits : 0;
  const int entry = a.tile_entry != nullptr ? a.tile_entry[tile] : tile;
  const int q0 = a.tile_entry != nullptr ? a.tile_q0[tile] : 0;
  const int kvh = blockIdx.y, group = a.q_heads / a.kv_heads, D = a.D, V = a.V, ps = a.page_size;
  const int tok0 = a.q_start[entry], q_len = a.q_start[entry + 1] - tok0;
  const int first_pos = a.kv_len[entry] - q_len;
  const int tokens = min(a.tile_tokens, q_len - q0), rows = tokens * group;
  const int* table = a.block_tables + (int64_t)entry * a.table_stride;
  if (tokens <= 0 || (int)blockIdx.z * KV_ROWS >= rows) return;

  const int row_lo = blockIdx.z * KV_ROWS + wave * 16;              // this wave's rows
  const bool wave_live = row_lo < rows;
  const int row = row_lo + col, my_row = min(row, rows - 1);
  const bool live = row < rows;
  const int t = my_row / group, head = kvh * group + my_row % group;
  const int pos = first_pos + q0 + t;
  // the tile's and the wave's first and last positions
  const int p_lo = first_pos + q0 + (int)blockIdx.z * KV_ROWS / group;
  const int p_hi = first_pos + q0 + min((int)blockIdx.z * KV_ROWS + KV_ROWS - 1, rows - 1) / group;
  const int w_lo = first_pos + q0 + min(row_lo, rows - 1) / group, w_hi = first_pos + q0 + min(row_lo + 15, rows - 1) / group;

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
  kv_f4 acc[2 * DC];
#pragma unroll
  for (int v = 0; v < 2 * DC; ++v) acc[v] = kv_f4{0.f, 0.f, 0.f, 0.f};
  const bool sink = a.sinks != nullptr && split == 0;
  float m_run = sink ? a.sinks[head] * LOG2E : -INFINITY;
  float l_run = sink && grp == 0 ? 1.f : 0.f;                       // (sums are lane by lane until the end)

  const int j_first = a.window > 0 ? max(0, p_lo - a.window + 1) : 0;
  const int b_end = p_hi >= 0 ? p_hi / KV_KEYS + 1 : 0;             // (a padding row has no keys)
  const int step = max(a.splits, 1);
  // this thread's key of a block and its first 16-byte piece of it
  const int k_row = tid >> 3, k_piece = tid & 7, pieces = D / 8;
  auto page_of = [&](int b) {                                        // (released or absent pages: any page will do)
    return max(table[min((b * KV_KEYS + k_row) / ps, a.table_stride - 1)], 0);
  };
  kv_u4 raw[CN];
  auto fetch = [&](int b, int page) {
    const bf16_t* kr = a.pages + (((int64_t)page * a.kv_heads + kvh) * ps + (b * KV_KEYS + k_row) % ps) * D;
#pragma unroll
    for (int n = 0; n < CN; ++n) {
      const int piece = k_piece + 8 * n;
      raw[n] = *reinterpret_cast<const kv_u4*>(kr + 8 * min(piece, pieces - 1));
      if (piece >= pieces) raw[n] = kv_u4{0, 0, 0, 0};
    }
  };
  auto put = [&](int buf) {
#pragma unroll
    for (int n = 0; n < CN; ++n) {
      const int piece = k_piece + 8 * n;
      if (piece < 4 * DC) *reinterpret_cast<kv_u4*>(&kt[buf][k_row * LD + 8 * piece]) = raw[n];
    }
  };
  int b = j_first / KV_KEYS + split;
  if (b < b_end) {
    fetch(b, page_of(b));
    put(0);
  }
  int page_next = page_of(min(b + step, max(b_end - 1, 0)));
  int buf = 0;
  __syncthreads();
  for (; b < b_end; b += step, buf ^= 1) {
    const bool more = b + step < b_end;
    if (more) fetch(b + step, page_next);
    page_next = page_of(min(b + 2 * step, b_end - 1));
    const int j0 = b * KV_KEYS;
    if (wave_live && j0 <= w_hi && (a.window <= 0 || j0 + KV_KEYS - 1 > w_lo - a.window)) {
      const bf16_t* kb = kt[buf];
      kv_f4 s[2] = {kv_f4{0.f, 0.f, 0.f, 0.f}, kv_f4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
      for (int d = 0; d < DC; ++d)
#pragma unroll
        for (int sub = 0; sub < 2; ++sub) {
          const kv_bf8 k8 = *reinterpret_cast<const kv_bf8*>(&kb[(16 * sub + col) * LD + 32 * d + 8 * grp]);
          s[sub] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k8, qb[d], s[sub], 0, 0, 0);
        }
      // s[sub][i]: key j0 + 16 sub + 4 grp + i against row `col`
      const bool whole = j0 + KV_KEYS - 1 <= w_lo && (a.window <= 0 || j0 > w_hi - a.window);
      float mx = -INFINITY;
#pragma unroll
      for (int sub = 0; sub < 2; ++sub)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          float x = s[sub][i] * scale2;
          if (!whole) {
            const int j = j0 + 16 * sub + 4 * grp + i;
            x = j <= pos && (a.window <= 0 || j > pos - a.window) ? x : -INFINITY;
          }
          s[sub][i] = x;
          mx = fmaxf(mx, x);
        }
      mx = fmaxf(mx, __shfl_xor(mx, 16, DLI_WAVE));
      mx = fmaxf(mx, __shfl_xor(mx, 32, DLI_WAVE));
      const float m_new = fmaxf(m_run, mx);
      const bool any = m_new > -INFINITY;
      const float alpha = any ? __builtin_amdgcn_exp2f(m_run - m_new) : 1.f;
      const bool moved = __any(m_new > m_run);
      float sum = 0.f;
      kv_bf8 pb;
#pragma unroll
      for (int sub = 0; sub < 2; ++sub)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float p = any ? __builtin_amdgcn_exp2f(s[sub][i] - m_new) : 0.f;
          sum += p;
          pb[4 * sub + i] = (bf16_t)p;
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
          const kv_bf4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((kv_lds4)(vb + 16 * v));
          const kv_bf4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((kv_lds4)(vb + 16 * LD + 16 * v));
          const kv_bf8 v8 = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
          acc[v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v8, pb, acc[v], 0, 0, 0);
        }
    }
    if (more) put(buf ^ 1);
    __syncthreads();
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
  return group >= KV_ROWS ? 1 : KV_ROWS / group;
}

// How many workgroups share an entry's keys in a step of single tokens: as many as bring the launch to two a
// compute unit, 32 at most. It depends on the heads and the number of entries, never on their lengths.
int dli_attention_keyvalue_splits(int q_heads, int kv_heads, int entries) {
  if (q_heads <= 0 || kv_heads <= 0 || q_heads % kv_heads != 0 || entries <= 0) return 1;
  const int group = q_heads / kv_heads;
  const int64_t workgroups = (int64_t)entries * kv_heads * ((group + KV_ROWS - 1) / KV_ROWS);
  const int64_t splits = 512 / workgroups;
  return splits < 1 ? 1 : splits > 32 ? 32 : (int)splits;
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
  const int group = q_heads / kv_heads;
  a.tile_tokens = tile_entry == nullptr ? 1 : dli_attention_keyvalue_tile_tokens(q_heads, kv_heads);
  const dim3 grid(tiles * splits, kv_heads, (a.tile_tokens * group + KV_ROWS - 1) / KV_ROWS);
  if (grid.z > 65535) return DLI_ERR_ARGUMENT;
  const int dc = (head_dim + 31) / 32;
#define KV_CASE(DC) attention_keyvalue_kernel<DC><<<grid, 256, 0, stream>>>(a)
  if (dc <= 1) KV_CASE(1);
  else if (dc == 2) KV_CASE(2);
  else if (dc == 3) KV_CASE(3);
  else if (dc == 4) KV_CASE(4);
  else if (dc == 5) KV_CASE(5);
  else if (dc == 6) KV_CASE(6);
  else if (dc <= 8) KV_CASE(8);
  else if (dc == 9) KV_CASE(9);
  else if (dc == 10) KV_CASE(10);
  else if (dc <= 12) KV_CASE(12);
  else if (dc <= 16) KV_CASE(16);
  else if (dc <= 18) KV_CASE(18);
  else KV_CASE(20);
#undef KV_CASE
  const int status = dli_launch_status();
  if (status != DLI_OK || splits == 1) return status;
  return dli_attention_scored_merge_bf16(parts, splits, tiles, q_heads, value_dim, out, out_stride, stream);
}

}  // extern "C"
