// Attention of grouped heads for the portions of a bfloat16 step, on the matrix cores, keys and values through LDS: a
// chunked mask, a window that may keep the first positions, a sink (of score 0 or of a score per head), values of another
// size than keys, value heads shared by several key heads, a sigmoid gate, an unrounded result. (A penalty on the distance,
// and sizes that this file does not take, are computed by csrc/attention_scored_mfma.hip.)
//
// A kv head's query heads read the same keys, so the rows of a tile are (token, query head) pairs: as many whole tokens of an
// entry as fit 64 rows (one token, 64 heads at a time, where a group is larger); a wave takes 16 of them. The tile's
// visible keys and their values pass through LDS in blocks of 64, read from memory once for all rows, the next block and the
// one after's page numbers in flight meanwhile. Both products run on v_mfma_f32_16x16x32_bf16 in transposed form, S^T = K Q^T and
// O^T = V^T P^T, so a lane holds scores of ONE row: of the keys 4 g + i and 16 + 4 g + i of a run of 32 (g = lane / 16,
// i < 4), which are the eight k of the second product as they stand. The pages keep a value's keys side by side; in
// LDS the eight keys of a lane lie next to each other, so that its other operand is one 16-byte read. Rows in LDS are
// padded by 16 bytes: sixteen rows' 16-byte pieces then lie in all 64 banks.
//
// Softmax with exp2 (log2 e in the scale), online, in 32-bit; P is rounded to bfloat16 for the second product while the running
// sum keeps the unrounded values, as in the other matrix-core attention.
#include "common.h"

typedef __bf16 ag_bf8 __attribute__((ext_vector_type(8)));
typedef __bf16 ag_bf4 __attribute__((ext_vector_type(4)));
typedef float ag_f4 __attribute__((ext_vector_type(4)));
typedef unsigned ag_u4 __attribute__((ext_vector_type(4)));
typedef unsigned ag_u2 __attribute__((ext_vector_type(2)));

#define AG_KEYS 64
#define AG_ROWS 64

struct GroupedArgs {
  const bf16_t* q; int64_t q_stride;
  const bf16_t* k_pages;                       // [pages][kv_heads][page_size][D]
  const bf16_t* v_pages;                       // [pages][v_heads][V][page_size]
  bf16_t* out; int64_t out_stride; float* out32;
  const int* q_start; const int* kv_len; const int* block_tables; int table_stride;
  const int* tile_entry; const int* tile_q0;
  int q_heads, kv_heads, v_heads, D, V, page_size, tile_tokens;
  float scale; int window, chunk, keep_first, sink;
  const float* sinks;
  const float* gate; int64_t gate_stride;
};

// The first position that `pos` sees, kept ones aside.
__device__ __forceinline__ int ag_low(const GroupedArgs& a, int pos) {
  int lo = a.chunk > 0 ? pos / a.chunk * a.chunk : 0;
  if (a.window > 0) lo = max(lo, pos - a.window + 1);
  return lo;
}

// Keys of up to 32 DC components, values of up to 16 VT.
template <int DC, int VT>
__global__ __launch_bounds__(256, 2) void attention_grouped_kernel(GroupedArgs a) {
  constexpr float LOG2E = 1.4426950408889634f;
  constexpr int LD = 32 * DC + 8, LV = AG_KEYS + 8;
  constexpr int CN = (4 * DC + 7) / 8, VN = (VT + 1) / 2;            // 16-byte pieces of a key, and of values, that a thread brings
  __shared__ __align__(16) bf16_t kt[2][AG_KEYS * LD], vt[2][16 * VT * LV];
  const int tid = threadIdx.x, lane = tid % 64, wave = __builtin_amdgcn_readfirstlane(tid / 64), col = lane & 15, grp = lane >> 4;
  const int tile = gridDim.x - 1 - blockIdx.x;                       // (a portion's last tiles see most keys)
  const int entry = a.tile_entry[tile], q0 = a.tile_q0[tile];
  const int kvh = blockIdx.y, vh = kvh % a.v_heads, group = a.q_heads / a.kv_heads, D = a.D, V = a.V, ps = a.page_size;
  const int tok0 = a.q_start[entry], q_len = a.q_start[entry + 1] - tok0;
  const int first_pos = a.kv_len[entry] - q_len;
  const int tokens = min(a.tile_tokens, q_len - q0), rows = tokens * group;
  const int* table = a.block_tables + (int64_t)entry * a.table_stride;
  const int z_lo = blockIdx.z * AG_ROWS;
  if (tokens <= 0 || z_lo >= rows) return;

  const int row_lo = z_lo + wave * 16;                               // this wave's rows
  const bool wave_live = row_lo < rows, live = row_lo + col < rows;
  const int mine = min(row_lo + col, rows - 1);
  const int t = mine / group, head = kvh * group + mine % group, pos = first_pos + q0 + t;
  // the tile's and the wave's first and last positions
  const int p_lo = first_pos + q0 + z_lo / group, p_hi = first_pos + q0 + min(z_lo + AG_ROWS - 1, rows - 1) / group;
  const int w_lo = first_pos + q0 + min(row_lo, rows - 1) / group;
  const int w_hi = first_pos + q0 + min(row_lo + 15, rows - 1) / group;
  const int my_chunk = a.chunk > 0 ? pos / a.chunk * a.chunk : 0, my_low = ag_low(a, pos);
  const int keep = a.window > 0 ? a.keep_first : 0;                  // keys below it are seen from any distance in the chunk
  const int w_low_lo = ag_low(a, w_lo), w_low_hi = ag_low(a, w_hi);

  ag_bf8 qb[DC];
  {
    const bf16_t* qr = a.q + (int64_t)(tok0 + q0 + t) * a.q_stride + (int64_t)head * D;
#pragma unroll
    for (int d = 0; d < DC; ++d) {
      const int at = 32 * d + 8 * grp;
      qb[d] = at < D ? *reinterpret_cast<const ag_bf8*>(qr + at) : ag_bf8{};
    }
  }
  const float scale2 = a.scale * LOG2E;
  const float not_seen = scale2 >= 0.f ? -INFINITY : INFINITY;       // times the scale: minus infinity
  ag_f4 acc[VT];
#pragma unroll
  for (int v = 0; v < VT; ++v) acc[v] = ag_f4{0.f, 0.f, 0.f, 0.f};
  const bool sink = a.sinks != nullptr || a.sink;
  float m_run = a.sinks != nullptr ? a.sinks[head] * LOG2E : sink ? 0.f : -INFINITY;
  float l_run = sink && grp == 0 ? 1.f : 0.f;                        // (sums are lane by lane until the end)

  const int b_first = ag_low(a, p_lo) / AG_KEYS, b_end = p_hi / AG_KEYS + 1;
  const int b_chunk = a.chunk > 0 ? p_lo / a.chunk * a.chunk / AG_KEYS : 0;
  const int b_keep = (keep + AG_KEYS - 1) / AG_KEYS;                 // blocks that hold kept keys
  auto after = [&](int b) { return b + 1 >= b_keep && b + 1 < b_first ? b_first : b + 1; };
  // this thread's keys of a block (k_row + 32 n) and its first 16-byte piece of each; its eight keys of value rows v_row + 32 n
  const int k_row = tid >> 3, k_piece = tid & 7, pieces = D / 8, v_row = tid >> 3, v_piece = tid & 7;
  int page_k[2], page_v;
  auto look = [&](int b) {                                           // (released or absent pages: any page will do)
#pragma unroll
    for (int n = 0; n < 2; ++n) page_k[n] = max(table[min((b * AG_KEYS + k_row + 32 * n) / ps, a.table_stride - 1)], 0);
    page_v = max(table[min((b * AG_KEYS + 8 * v_piece) / ps, a.table_stride - 1)], 0);
  };
  ag_u4 raw_k[2][CN], raw_v[VN];
  auto fetch = [&](int b) {
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      const bf16_t* kr = a.k_pages + (((int64_t)page_k[n] * a.kv_heads + kvh) * ps + (b * AG_KEYS + k_row + 32 * n) % ps) * D;
#pragma unroll
      for (int c = 0; c < CN; ++c) {
        const int piece = k_piece + 8 * c;
        raw_k[n][c] = *reinterpret_cast<const ag_u4*>(kr + 8 * min(piece, pieces - 1));
        if (piece >= pieces) raw_k[n][c] = ag_u4{0, 0, 0, 0};
      }
    }
    const bf16_t* vr = a.v_pages + ((int64_t)page_v * a.v_heads + vh) * V * ps + (b * AG_KEYS + 8 * v_piece) % ps;
#pragma unroll
    for (int n = 0; n < VN; ++n) raw_v[n] = *reinterpret_cast<const ag_u4*>(vr + (int64_t)min(v_row + 32 * n, V - 1) * ps);
  };
  auto put = [&](int buf) {
#pragma unroll
    for (int n = 0; n < 2; ++n)
#pragma unroll
      for (int c = 0; c < CN; ++c) {
        const int piece = k_piece + 8 * c;
        if (piece < 4 * DC) *reinterpret_cast<ag_u4*>(&kt[buf][(k_row + 32 * n) * LD + 8 * piece]) = raw_k[n][c];
      }
    // keys 8 p .. 8 p + 7 of a run of 32 go to the places of lane groups 2 (p % 2) and the next, half p / 2 of each
    const int at = 32 * (v_piece / 4) + 16 * (v_piece % 2) + 4 * (v_piece % 4 / 2);
#pragma unroll
    for (int n = 0; n < VN; ++n)
      if (v_row + 32 * n < 16 * VT) {
        bf16_t* to = &vt[buf][(v_row + 32 * n) * LV + at];
        *reinterpret_cast<ag_u2*>(to) = ag_u2{raw_v[n][0], raw_v[n][1]};
        *reinterpret_cast<ag_u2*>(to + 8) = ag_u2{raw_v[n][2], raw_v[n][3]};
      }
  };
  int b = keep > 0 && b_chunk < b_keep ? min(b_chunk, b_first) : b_first;
  look(b);
  fetch(b);
  put(0);
  int next = after(b);
  look(min(next, b_end - 1));
  int buf = 0;
  __syncthreads();
  for (; b < b_end; buf ^= 1) {
    const bool more = next < b_end;
    if (more) {
      fetch(next);
      look(min(after(next), b_end - 1));
    }
    const int j0 = b * AG_KEYS;
    if (wave_live && j0 <= w_hi && (j0 + AG_KEYS - 1 >= w_low_lo || j0 < keep)) {
      const bf16_t* kb = kt[buf];
      ag_f4 s[4];
#pragma unroll
      for (int sub = 0; sub < 4; ++sub) s[sub] = ag_f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int d = 0; d < DC; ++d)
#pragma unroll
        for (int sub = 0; sub < 4; ++sub)
          s[sub] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              *reinterpret_cast<const ag_bf8*>(&kb[(16 * sub + col) * LD + 32 * d + 8 * grp]), qb[d], s[sub], 0, 0, 0);
      // s[sub][i]: key j0 + 16 sub + 4 grp + i against row `col`
      if (j0 + AG_KEYS - 1 > w_lo || j0 < w_low_hi) {                // (else every key is seen by every row)
#pragma unroll
        for (int sub = 0; sub < 4; ++sub)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int j = j0 + 16 * sub + 4 * grp + i;
            s[sub][i] = j <= pos && (j >= my_low || (j < keep && j >= my_chunk)) ? s[sub][i] : not_seen;
          }
      }
      // (the largest score is the largest product for a positive scale, the smallest for a negative one)
      float mx = not_seen;
#pragma unroll
      for (int sub = 0; sub < 4; ++sub)
#pragma unroll
        for (int i = 0; i < 4; ++i) mx = scale2 >= 0.f ? fmaxf(mx, s[sub][i]) : fminf(mx, s[sub][i]);
      mx *= scale2;
      mx = fmaxf(mx, __shfl_xor(mx, 16, DLI_WAVE));
      mx = fmaxf(mx, __shfl_xor(mx, 32, DLI_WAVE));
      const float m_new = fmaxf(m_run, mx);
      const float m_safe = m_new > -INFINITY ? m_new : 0.f;          // (nothing seen yet: every weight is exp2(-inf))
      const float alpha = __builtin_amdgcn_exp2f(m_run - m_safe);
      const bool moved = __any(m_new > m_run);
      float sum = 0.f;
      ag_bf8 pb[2];
#pragma unroll
      for (int sub = 0; sub < 4; ++sub)
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
        for (int v = 0; v < VT; ++v) acc[v] *= alpha;
      }
      const bf16_t* vb = vt[buf] + col * LV + 8 * grp;
#pragma unroll
      for (int v = 0; v < VT; ++v)
#pragma unroll
        for (int k = 0; k < 2; ++k)
          acc[v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const ag_bf8*>(vb + 16 * v * LV + 32 * k), pb[k], acc[v], 0, 0, 0);
    }
    if (more) put(buf ^ 1);
    __syncthreads();
    b = next;
    next = after(next);
  }
  float l = l_run + __shfl_xor(l_run, 16, DLI_WAVE);
  l += __shfl_xor(l, 32, DLI_WAVE);
  if (!live) return;
  const float inv = l > 0.f ? 1.f / l : 0.f;
  // acc[v][i] is value 16 v + 4 grp + i of this lane's row
  const int64_t row = tok0 + q0 + t;
#pragma unroll
  for (int v = 0; v < VT; ++v)
    if (16 * v + 4 * grp < V) {
      const int64_t at = (int64_t)head * V + 16 * v + 4 * grp;
      ag_f4 y = acc[v] * inv;
      if (a.gate != nullptr)
#pragma unroll
        for (int i = 0; i < 4; ++i) y[i] *= 1.f / (1.f + __expf(-a.gate[row * a.gate_stride + at + i]));
      if (a.out32 != nullptr) {
        *reinterpret_cast<ag_f4*>(a.out32 + row * a.out_stride + at) = y;
      } else {
        ag_bf4 o;
#pragma unroll
        for (int i = 0; i < 4; ++i) o[i] = (bf16_t)y[i];
        *reinterpret_cast<ag_bf4*>(a.out + row * a.out_stride + at) = o;
      }
    }
}

template <int DC>
static int launch_grouped(const GroupedArgs& a, const dim3& grid, hipStream_t stream) {
#define VCASE(VT) case VT: attention_grouped_kernel<DC, VT><<<grid, 256, 0, stream>>>(a); break;
  switch ((a.V + 15) / 16) {
    VCASE(1) VCASE(2) VCASE(3) VCASE(4) VCASE(5) VCASE(6)
    case 7: VCASE(8)
    default: return DLI_ERR_ARGUMENT;
  }
#undef VCASE
  return dli_launch_status();
}

extern "C" {

int dli_attention_grouped_supports(int head_dim, int value_dim, int page_size) {
  return head_dim >= 8 && head_dim <= 128 && head_dim % 8 == 0 && value_dim >= 4 && value_dim <= 128 && value_dim % 4 == 0 &&
         page_size > 0 && page_size % 8 == 0;
}

// Whole tokens of a tile (the host builds its tile list with this).
int dli_attention_grouped_tile_tokens(int q_heads, int kv_heads) {
  if (q_heads <= 0 || kv_heads <= 0 || q_heads % kv_heads != 0) return DLI_ERR_ARGUMENT;
  const int group = q_heads / kv_heads;
  return group >= AG_ROWS ? 1 : AG_ROWS / group;
}

int dli_attention_grouped(const void* q, int64_t q_stride, const void* k_pages, const void* v_pages, void* out, int64_t out_stride,
                          const int* q_start, const int* kv_len, const int* block_tables, int table_stride, const int* tile_entry,
                          const int* tile_q0, int tiles, int q_heads, int kv_heads, int v_heads, int head_dim, int value_dim,
                          int page_size, float scale, int window, int chunk, int keep_first, int sink, const float* sinks,
                          const float* gate, int64_t gate_stride, int out_is_f32, hipStream_t stream) {
  if (tiles <= 0) return DLI_OK;
  if (!dli_attention_grouped_supports(head_dim, value_dim, page_size) || q_heads <= 0 || kv_heads <= 0 || q_heads % kv_heads ||
      v_heads <= 0 || kv_heads % v_heads || kv_heads > 65535 || table_stride <= 0 || window < 0 || chunk < 0 || keep_first < 0 ||
      tile_entry == nullptr || tile_q0 == nullptr || q_stride % 8 || out_stride % 4 ||
      ((uintptr_t)q | (uintptr_t)k_pages | (uintptr_t)v_pages | (uintptr_t)out) % 16)
    return DLI_ERR_ARGUMENT;
  GroupedArgs a;
  a.q = (const bf16_t*)q; a.q_stride = q_stride; a.k_pages = (const bf16_t*)k_pages; a.v_pages = (const bf16_t*)v_pages;
  a.out = (bf16_t*)out; a.out_stride = out_stride; a.out32 = out_is_f32 ? (float*)out : nullptr; a.q_start = q_start; a.kv_len = kv_len;
  a.block_tables = block_tables; a.table_stride = table_stride; a.tile_entry = tile_entry; a.tile_q0 = tile_q0; a.q_heads = q_heads;
  a.kv_heads = kv_heads; a.v_heads = v_heads; a.D = head_dim; a.V = value_dim; a.page_size = page_size; a.scale = scale;
  a.window = window; a.chunk = chunk; a.keep_first = keep_first; a.sink = sink; a.sinks = sinks; a.gate = gate; a.gate_stride = gate_stride;
  a.tile_tokens = dli_attention_grouped_tile_tokens(q_heads, kv_heads);
  const int group = q_heads / kv_heads;
  const dim3 grid(tiles, kv_heads, (a.tile_tokens * group + AG_ROWS - 1) / AG_ROWS);
  switch ((head_dim + 31) / 32) {
    case 1: return launch_grouped<1>(a, grid, stream);
    case 2: return launch_grouped<2>(a, grid, stream);
    case 3: return launch_grouped<3>(a, grid, stream);
    default: return launch_grouped<4>(a, grid, stream);
  }
}

}  // extern "C"
