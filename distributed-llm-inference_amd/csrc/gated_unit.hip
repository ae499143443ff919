// A gated linear recurrence per channel (a real-gated recurrent unit) whose two gates are block-diagonal maps of
// its own input. With u the input of a token (C channels in `blocks` equal parts of s), and for block b
//   r = sigmoid(Wr[b] u_b + br),  i = sigmoid(Wi[b] u_b + bi),  a = exp(-r decay),  decay >= 0 per channel:
//   S <- a S + sqrt(1 - a^2) i u,   out = S * gelu(y + y_bias)   (gelu in its tanh form)
// S is float32 [C] at the start of the request's state slot and starts from zeros where the entry's first row has
// position 0. Everything is 32-bit: sqrt(1 - a^2) is sqrt(-expm1(-2 r decay)), and the gates' products take u
// unrounded; where the weights are bfloat16 they run on the bfloat16 matrix cores with u as the sum of
// three bfloat16 numbers (24 bits: u itself), the products' sums in 32-bit.
//
// Steps with portions, 64 tokens of an entry (a tile) at a time:
//   gates    a wave takes a tile and 32 channels of a block: both gates' products, a and the input, and the tile's
//            recurrence from zero as a scan: in a lane over four tokens, over the four lane groups, over the four
//            16-token parts. It leaves S_local and the product P of the a's up to each token, and the tile's end.
//   carry    a thread a channel walks an entry's tiles: what the state is when each begins, and after the last
//   apply    out = (S_local + P * carry) * gelu(y + y_bias)
// Steps of single tokens: one launch, the recurrence's step where the gates are made.
// Weights that are not bfloat16, or parts whose size is no multiple of 8, take vector-unit kernels, any size.
#include "common.h"

typedef __bf16 gu_bf8 __attribute__((ext_vector_type(8)));
typedef float gu_f4 __attribute__((ext_vector_type(4)));

#define GU_TILE 64

struct GuArgs {
  const float* u; int64_t u_stride;            // [rows][C]
  const void* wr; const void* wi;              // [blocks][s][s], a row an output
  const float* br; const float* bi;            // [C]
  const float* decay;                          // [C]
  const float* y; int64_t y_stride; const float* y_bias;
  float* state; int64_t state_stride;
  const int* q_start; const int* positions; const int* state_slots;
  const int* tile_entry; const int* tile_q0;   // nullptr: every entry is one row
  float* s_local; float* p_local;              // [rows][C]
  float* ends;                                 // [tiles][2][C]: P and S at a tile's end; the carry kernel puts the
                                               // state at a tile's beginning in place of the first
  void* out; int64_t out_stride;
  int rows, entries, C, s, blocks;
};

// (the hardware's exp2, reciprocal and square root are good to an ulp or so; the step is held by their number)
__device__ __forceinline__ float gu_sigmoid(float x) { return __builtin_amdgcn_rcpf(1.f + __expf(-x)); }
__device__ __forceinline__ float gu_gelu(float z) {
  return z * gu_sigmoid(1.5957691216057308f * (z + 0.044715f * z * z * z));      // 2 sqrt(2 / pi)
}
// a and the recurrence's input from the gates' pre-activations. 1 - a^2 = 1 - exp(-t), t = 2 r decay: near t = 0 by its
// Taylor series (the next term is below 2e-8 of the sum at t = 1/4), where a^2 would lose what is left of it.
__device__ __forceinline__ void gu_gates(float r_pre, float i_pre, float u, float decay, float* a, float* in) {
  const float x = gu_sigmoid(r_pre) * decay, t = 2.f * x;
  *a = __expf(-x);
  const float series = t * (1.f - t * (1.f / 2) * (1.f - t * (1.f / 3) * (1.f - t * (1.f / 4) * (1.f - t * (1.f / 5) *
                       (1.f - t * (1.f / 6) * (1.f - t * (1.f / 7)))))));
  const float rest = t < 0.25f ? series : fmaf(-*a, *a, 1.f);
  *in = __builtin_amdgcn_sqrtf(rest) * gu_sigmoid(i_pre) * u;
}

// What a single token's step at channel c reads besides the gates, asked for before they are made.
struct GuSingle {
  float u, y, old;
  float* state;
  bool fresh;
};
__device__ __forceinline__ GuSingle gu_single_read(const GuArgs& p, int row, int c) {
  GuSingle x;
  x.u = p.u[(int64_t)row * p.u_stride + c];
  x.y = p.y[(int64_t)row * p.y_stride + c];
  x.state = p.state + (int64_t)p.state_slots[row] * p.state_stride + c;
  x.old = *x.state;
  x.fresh = p.positions[row] == 0;
  return x;
}
template <typename T>
__device__ __forceinline__ void gu_single_step(const GuArgs& p, const GuSingle& x, int row, int c, float r_pre, float i_pre) {
  float a, in;
  gu_gates(r_pre + p.br[c], i_pre + p.bi[c], x.u, p.decay[c], &a, &in);
  const float S = fmaf(a, x.fresh ? 0.f : x.old, in);
  *x.state = S;
  ((T*)p.out)[(int64_t)row * p.out_stride + c] = from_f32<T>(S * gu_gelu(x.y + (p.y_bias != nullptr ? p.y_bias[c] : 0.f)));
}

// Eight floats as the sum of three bfloat16 vectors.
__device__ __forceinline__ void gu_split(const float* x, gu_bf8 h[3]) {
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    const bf16_t a = (bf16_t)x[e];
    const float r1 = x[e] - (float)a;
    const bf16_t b = (bf16_t)r1;
    h[0][e] = a;
    h[1][e] = b;
    h[2][e] = (bf16_t)(r1 - (float)b);
  }
}

// TB parts of 16 tokens x NC of 16 channels a wave; SINGLE: rows are entries (TB 1).
template <int TB, int NC, int WAVES, bool SINGLE>
__global__ __launch_bounds__(64 * WAVES) void gated_unit_mfma_kernel(GuArgs p) {
  const int lane = threadIdx.x % 64, wave = threadIdx.x / 64, col = lane & 15, grp = lane >> 4;
  const int s = p.s, per_block = (s + 16 * NC - 1) / (16 * NC);
  const int group = blockIdx.y * WAVES + wave;
  if (group >= p.blocks * per_block) return;
  const int block = group / per_block, n0 = (group % per_block) * 16 * NC;   // first output within the block
  int row0, n_rows;
  if constexpr (SINGLE) {
    row0 = blockIdx.x * 16;
    n_rows = min(16, p.rows - row0);
  } else {
    const int entry = p.tile_entry[blockIdx.x], q0 = p.tile_q0[blockIdx.x];
    row0 = p.q_start[entry] + q0;
    n_rows = min(GU_TILE, p.q_start[entry + 1] - row0);
  }
  if (n_rows <= 0) return;
  const bf16_t* wr[NC];
  const bf16_t* wi[NC];
#pragma unroll
  for (int n = 0; n < NC; ++n) {
    const int64_t at = ((int64_t)block * s + min(n0 + 16 * n + col, s - 1)) * s;
    wr[n] = (const bf16_t*)p.wr + at;
    wi[n] = (const bf16_t*)p.wi + at;
  }
  gu_f4 ar[TB][NC], ai[TB][NC];
#pragma unroll
  for (int t = 0; t < TB; ++t)
#pragma unroll
    for (int n = 0; n < NC; ++n) ar[t][n] = ai[t][n] = gu_f4{0.f, 0.f, 0.f, 0.f};
  GuSingle single[SINGLE ? 4 : 1][SINGLE ? NC : 1];
  if constexpr (SINGLE) {
#pragma unroll
    for (int n = 0; n < NC; ++n)
#pragma unroll
      for (int i = 0; i < 4; ++i)               // (rows and outputs past the last are the last again; nothing is stored for them)
        single[i][n] = gu_single_read(p, row0 + min(4 * grp + i, n_rows - 1), block * s + min(n0 + 16 * n + col, s - 1));
  }
  // KU steps of 32 k are asked for at once, and the next KU before these are multiplied
  constexpr int KU = SINGLE ? 4 : 1;
  struct Operands { gu_bf8 r[KU][NC], i[KU][NC]; gu_f4 u[KU][TB][2]; };
  const float* ur[TB];
#pragma unroll
  for (int t = 0; t < TB; ++t) ur[t] = p.u + (int64_t)(row0 + min(16 * t + col, n_rows - 1)) * p.u_stride + (int64_t)block * s;
  auto fetch = [&](Operands& o, int k0) {
#pragma unroll
    for (int j = 0; j < KU; ++j) {
      const int k = k0 + 32 * j + 8 * grp, at = k < s ? k : 0;   // (s is a multiple of 8; what lies past it counts as zero)
#pragma unroll
      for (int n = 0; n < NC; ++n) {
        o.r[j][n] = *reinterpret_cast<const gu_bf8*>(wr[n] + at);
        o.i[j][n] = *reinterpret_cast<const gu_bf8*>(wi[n] + at);
      }
#pragma unroll
      for (int t = 0; t < TB; ++t)
#pragma unroll
        for (int e = 0; e < 2; ++e) o.u[j][t][e] = *reinterpret_cast<const gu_f4*>(ur[t] + at + 4 * e);
    }
  };
  auto multiply = [&](const Operands& o, int k0) {
#pragma unroll
    for (int j = 0; j < KU; ++j) {
      const bool in = k0 + 32 * j + 8 * grp < s;
      if (KU > 1 && k0 + 32 * j >= s) break;
#pragma unroll
      for (int t = 0; t < TB; ++t) {
        float x[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = in ? o.u[j][t][e / 4][e % 4] : 0.f;
        gu_bf8 h[3];
        gu_split(x, h);
#pragma unroll
        for (int q = 2; q >= 0; --q)            // the small parts first
#pragma unroll
          for (int n = 0; n < NC; ++n) {
            ar[t][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(h[q], o.r[j][n], ar[t][n], 0, 0, 0);
            ai[t][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(h[q], o.i[j][n], ai[t][n], 0, 0, 0);
          }
      }
    }
  };
  {
    Operands o0, o1;
    fetch(o0, 0);
    for (int k0 = 0; k0 < s; k0 += 64 * KU) {
      fetch(o1, k0 + 32 * KU);
      multiply(o0, k0);
      if (k0 + 32 * KU >= s) break;
      fetch(o0, k0 + 64 * KU);
      multiply(o1, k0 + 32 * KU);
    }
  }
  // ar[t][n][i]: token 16 t + 4 grp + i, output n0 + 16 n + col
#pragma unroll
  for (int n = 0; n < NC; ++n) {
    const int o = n0 + 16 * n + col;
    const bool live = o < s;
    const int c = block * s + min(o, s - 1);
    if constexpr (SINGLE) {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (live && 4 * grp + i < n_rows) 
          gu_single_step<bf16_t>(p, single[i][n], row0 + 4 * grp + i, c, ar[0][n][i], ai[0][n][i]);
    } else {
      const float cr = p.br[c], ci = p.bi[c], decay = p.decay[c];
      float P0 = 1.f, S0 = 0.f;                 // at the beginning of this part of 16 tokens
#pragma unroll
      for (int t = 0; t < TB; ++t) {
        float a[4], b[4];
        float A = 1.f, B = 0.f;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int tok = 16 * t + 4 * grp + i;
          const float u = p.u[(int64_t)(row0 + min(tok, n_rows - 1)) * p.u_stride + c];
          gu_gates(ar[t][n][i] + cr, ai[t][n][i] + ci, u, decay, &a[i], &b[i]);
          if (tok >= n_rows) { a[i] = 1.f; b[i] = 0.f; }
          A *= a[i];
          B = fmaf(a[i], B, b[i]);
        }
        // inclusive scan over the four lane groups: first by one group, then by two
#pragma unroll
        for (int d = 16; d <= 32; d <<= 1) {
          const float A1 = __shfl_up(A, d, DLI_WAVE), B1 = __shfl_up(B, d, DLI_WAVE);
          if (lane >= d) {
            B = fmaf(A, B1, B);
            A *= A1;
          }
        }
        float Ax = __shfl_up(A, 16, DLI_WAVE), Bx = __shfl_up(B, 16, DLI_WAVE);
        if (grp == 0) { Ax = 1.f; Bx = 0.f; }
        float P = P0 * Ax, S = fmaf(Ax, S0, Bx);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          P *= a[i];
          S = fmaf(a[i], S, b[i]);
          const int tok = 16 * t + 4 * grp + i;
          if (live && tok < n_rows) {
            p.s_local[(int64_t)(row0 + tok) * p.C + c] = S;
            p.p_local[(int64_t)(row0 + tok) * p.C + c] = P;
          }
        }
        P0 = __shfl(P, 48 + col, DLI_WAVE);
        S0 = __shfl(S, 48 + col, DLI_WAVE);
      }
      if (live && grp == 0) {
        p.ends[((int64_t)blockIdx.x * 2) * p.C + c] = P0;
        p.ends[((int64_t)blockIdx.x * 2 + 1) * p.C + c] = S0;
      }
    }
  }
}

// Any size, any type: a workgroup takes 16 outputs of a block and 16 rows at a time (thread: tx output, ty row), a tile's
// four sixteens one after the other; the scan by one thread an output.
#define GU_BK 32
template <typename T, bool SINGLE>
__global__ __launch_bounds__(256) void gated_unit_any_kernel(GuArgs p) {
  __shared__ float us[16][GU_BK + 1], rs[16][GU_BK + 1], is[16][GU_BK + 1], as[16][17], bs[16][17];
  const int tid = threadIdx.x, tx = tid % 16, ty = tid / 16;
  const int s = p.s, per_block = (s + 15) / 16;
  const int block = blockIdx.y / per_block, n0 = (blockIdx.y % per_block) * 16;
  int row0, n_rows;
  if constexpr (SINGLE) {
    row0 = blockIdx.x * 16;
    n_rows = min(16, p.rows - row0);
  } else {
    const int entry = p.tile_entry[blockIdx.x], q0 = p.tile_q0[blockIdx.x];
    row0 = p.q_start[entry] + q0;
    n_rows = min(GU_TILE, p.q_start[entry + 1] - row0);
  }
  const T* wr = (const T*)p.wr + (int64_t)block * s * s;
  const T* wi = (const T*)p.wi + (int64_t)block * s * s;
  const int o = n0 + tx;
  const int c = block * s + min(o, s - 1);
  float P = 1.f, S = 0.f;                       // (of the threads that scan)
  for (int t0 = 0; t0 < n_rows; t0 += 16) {
    float ar = 0.f, ai = 0.f;
    for (int k0 = 0; k0 < s; k0 += GU_BK) {
      __syncthreads();
      for (int idx = tid; idx < 16 * GU_BK; idx += 256) {
        const int r = idx / GU_BK, k = k0 + idx % GU_BK;
        const bool in = k < s;
        us[r][idx % GU_BK] = in && t0 + r < n_rows ? p.u[(int64_t)(row0 + t0 + r) * p.u_stride + (int64_t)block * s + k] : 0.f;
        rs[r][idx % GU_BK] = in && n0 + r < s ? to_f32(wr[(int64_t)(n0 + r) * s + k]) : 0.f;
        is[r][idx % GU_BK] = in && n0 + r < s ? to_f32(wi[(int64_t)(n0 + r) * s + k]) : 0.f;
      }
      __syncthreads();
#pragma unroll
      for (int k = 0; k < GU_BK; ++k) {
        ar = fmaf(us[ty][k], rs[tx][k], ar);
        ai = fmaf(us[ty][k], is[tx][k], ai);
      }
    }
    const bool live = o < s && t0 + ty < n_rows;
    if constexpr (SINGLE) {
      if (live) gu_single_step<T>(p, gu_single_read(p, row0 + ty, c), row0 + ty, c, ar, ai);
    } else {
      float a = 1.f, b = 0.f;
      if (live)
        gu_gates(ar + p.br[c], ai + p.bi[c], p.u[(int64_t)(row0 + t0 + ty) * p.u_stride + c], p.decay[c], &a, &b);
      as[ty][tx] = a;
      bs[ty][tx] = b;
      __syncthreads();
      if (ty == 0 && o < s)
        for (int r = 0; r < min(16, n_rows - t0); ++r) {
          P *= as[r][tx];
          S = fmaf(as[r][tx], S, bs[r][tx]);
          p.s_local[(int64_t)(row0 + t0 + r) * p.C + c] = S;
          p.p_local[(int64_t)(row0 + t0 + r) * p.C + c] = P;
        }
    }
  }
  if constexpr (!SINGLE)
    if (ty == 0 && o < s) {
      p.ends[((int64_t)blockIdx.x * 2) * p.C + c] = P;
      p.ends[((int64_t)blockIdx.x * 2 + 1) * p.C + c] = S;
    }
}

// A thread a channel of the entry that a tile with tile_q0 0 begins.
__global__ void gated_unit_carry_kernel(GuArgs p) {
  const int first = blockIdx.x, c = blockIdx.y * blockDim.x + threadIdx.x;
  if (p.tile_q0[first] != 0 || c >= p.C) return;
  const int entry = p.tile_entry[first];
  const int row0 = p.q_start[entry], tiles = (p.q_start[entry + 1] - row0 + GU_TILE - 1) / GU_TILE;
  float* st = p.state + (int64_t)p.state_slots[entry] * p.state_stride + c;
  const float old = *st;
  float S = p.positions[row0] == 0 ? 0.f : old;
  float* e = p.ends + (int64_t)first * 2 * p.C + c;
  constexpr int N = 16;                         // tiles asked for at once, the next ones before these are walked
  float P[2][N], E[2][N];
  auto fetch = [&](int w, int t0) {
#pragma unroll
    for (int j = 0; j < N; ++j) {               // (tiles past the last repeat it)
      const int64_t at = (int64_t)min(t0 + j, tiles - 1) * 2 * p.C;
      P[w][j] = e[at];
      E[w][j] = e[at + p.C];
    }
  };
  auto walk = [&](int w, int t0) {
#pragma unroll
    for (int j = 0; j < N; ++j)
      if (t0 + j < tiles) {
        e[(int64_t)(t0 + j) * 2 * p.C] = S;
        S = fmaf(P[w][j], S, E[w][j]);
      }
  };
  fetch(0, 0);
  for (int t0 = 0; t0 < tiles; t0 += 2 * N) {
    // (what is fetched ahead lies past what is being written: a tile's P is read before its place is taken)
    if (t0 + N < tiles) fetch(1, t0 + N);
    walk(0, t0);
    if (t0 + N >= tiles) break;
    if (t0 + 2 * N < tiles) fetch(0, t0 + 2 * N);
    walk(1, t0 + N);
  }
  *st = S;
}

template <typename T>
__global__ __launch_bounds__(256) void gated_unit_apply_kernel(GuArgs p) {
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= p.C) return;
  const int entry = p.tile_entry[blockIdx.x];
  const int row0 = p.q_start[entry] + p.tile_q0[blockIdx.x], end = min(row0 + GU_TILE, p.q_start[entry + 1]);
  const float carry = p.ends[(int64_t)blockIdx.x * 2 * p.C + c];
  const float yb = p.y_bias != nullptr ? p.y_bias[c] : 0.f;
  const int from = row0 + blockIdx.z * 8;
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    const int row = min(from + j, end - 1);     // (rows past the last are the last again)
    const float S = fmaf(p.p_local[(int64_t)row * p.C + c], carry, p.s_local[(int64_t)row * p.C + c]);
    const float v = S * gu_gelu(p.y[(int64_t)row * p.y_stride + c] + yb);
    if (from + j < end) ((T*)p.out)[(int64_t)row * p.out_stride + c] = from_f32<T>(v);
  }
}

extern "C" {

int dli_gated_unit_tile_rows() { return GU_TILE; }

// tile_entry == nullptr: a step of single tokens (rows == entries; s_local, p_local and ends are not used). Else the
// tiles of dli_gated_unit_tile_rows() rows of every entry, by entry and then by row; scratch s_local, p_local float
// [rows][C] and ends float [tiles][2][C].
int dli_gated_unit(const float* u, int64_t u_stride, const void* wr, const void* wi, const float* br, const float* bi,
                   const float* decay, const float* y, int64_t y_stride, const float* y_bias, float* state,
                   int64_t state_stride, const int* q_start, const int* positions, const int* state_slots,
                   const int* tile_entry, const int* tile_q0, int tiles, float* s_local, float* p_local, float* ends,
                   void* out, int64_t out_stride, int entries, int rows, int C, int blocks, int is_bf16, hipStream_t stream) {
  if (rows <= 0 || entries <= 0) return DLI_OK;
  const bool single = tile_entry == nullptr;
  if (C <= 0 || blocks <= 0 || C % blocks || u_stride < C || y_stride < C || out_stride < C || state_stride < C ||
      (single ? rows != entries : tiles <= 0 || tile_q0 == nullptr || s_local == nullptr || p_local == nullptr || ends == nullptr))
    return DLI_ERR_ARGUMENT;
  GuArgs p;
  p.u = u; p.u_stride = u_stride; p.wr = wr; p.wi = wi; p.br = br; p.bi = bi; p.decay = decay; p.y = y; p.y_stride = y_stride;
  p.y_bias = y_bias; p.state = state; p.state_stride = state_stride; p.q_start = q_start; p.positions = positions;
  p.state_slots = state_slots; p.tile_entry = tile_entry; p.tile_q0 = tile_q0; p.s_local = s_local; p.p_local = p_local;
  p.ends = ends; p.out = out; p.out_stride = out_stride; p.rows = rows; p.entries = entries; p.C = C; p.s = C / blocks;
  p.blocks = blocks;
  const int s = p.s;
  const bool mfma = is_bf16 && s % 8 == 0 && u_stride % 4 == 0 && ((uintptr_t)u | (uintptr_t)wr | (uintptr_t)wi) % 16 == 0;
  const int64_t g16 = (int64_t)blocks * ((s + 15) / 16), g32 = (int64_t)blocks * ((s + 31) / 32);
  if (g16 > 65535) return DLI_ERR_ARGUMENT;
  if (single) {
    const dim3 grid((rows + 15) / 16, (unsigned)g16);
    if (mfma) gated_unit_mfma_kernel<1, 1, 1, true><<<grid, 64, 0, stream>>>(p);
    else if (is_bf16) gated_unit_any_kernel<bf16_t, true><<<grid, 256, 0, stream>>>(p);
    else gated_unit_any_kernel<float, true><<<grid, 256, 0, stream>>>(p);
    return dli_launch_status();
  }
  if (mfma) gated_unit_mfma_kernel<4, 2, 4, false><<<dim3(tiles, (unsigned)((g32 + 3) / 4)), 256, 0, stream>>>(p);
  else if (is_bf16) gated_unit_any_kernel<bf16_t, false><<<dim3(tiles, (unsigned)g16), 256, 0, stream>>>(p);
  else gated_unit_any_kernel<float, false><<<dim3(tiles, (unsigned)g16), 256, 0, stream>>>(p);
  if (dli_launch_status() != DLI_OK) return DLI_ERR_LAUNCH;
  gated_unit_carry_kernel<<<dim3(tiles, (C + 63) / 64), 64, 0, stream>>>(p);
  if (dli_launch_status() != DLI_OK) return DLI_ERR_LAUNCH;
  const dim3 grid(tiles, (C + 255) / 256, GU_TILE / 8);
  if (is_bf16) gated_unit_apply_kernel<bf16_t><<<grid, 256, 0, stream>>>(p);
  else gated_unit_apply_kernel<float><<<grid, 256, 0, stream>>>(p);
  return dli_launch_status();
}

}  // extern "C"
