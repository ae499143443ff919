// Feed-forward layers beyond the gated product: a polynomial activation with norms, and a mixture of
// small experts with a router. T is the type of what the matrix products read and write (float on the
// 32-bit path, bf16 when serving); statistics, the router and every sum are 32-bit.
//
//   poly_norm        out(T) = a N(z) + b N(z^2) + c N(z^3) + e, powers element by element, N(x) = x / sqrt(mean(x^2) + eps)
//                    over the row; z is the 32-bit result of the product before it
//   clamped_glu      y = g sigmoid(alpha g) (u + shift), g = min(gate, limit), u = clamp(up, -limit, limit); an infinite
//                    limit, alpha 1 and shift 0 give the plain silu(gate) * up
//   gelu_glu         y = gelu(gate) * up, tanh form (the same kernels)
//   router_choose    softmax over all router outputs, or the sigmoid of each; choice = score + correction; only the
//                    `keep` groups of neighbours with the largest best choice stay; the `top` largest choices; weights =
//                    the chosen scores (without correction) / (their sum + 1e-20) * scale, or scores * scale alone
//   expert_sort      the (token, choice) slots of real experts in runs by expert, and the list of row tiles
//   expert_up/down   the experts' products over those tiles (on the matrix cores for bfloat16 and sizes that are
//                    multiples of 32, else on the vector units, any size), the clamped activation between
//                    them; the down product leaves each slot's 32-bit result in the slot's own row. Where a slot's
//                    weight belongs on the expert's input, the up kernels multiply their 32-bit sums by it
//   expert_combine   out = sum_j w_j (expert j's result, or the input itself for an identity expert)
//                    + sigmoid(shared gate) * shared expert's result
//
// A row's result never depends on its place in a tile or on the other rows: every output sums its k in
// ascending order.
#include "common.h"

__global__ void poly_norm_kernel_f32in(const float* __restrict__ z, int64_t z_stride, const float* __restrict__ coef,
                                       void* __restrict__ out_, int64_t out_stride, int ff, float eps, int out_is_bf16) {
  __shared__ float scratch[3][16];
  const int64_t row = blockIdx.x;
  const float* zr = z + row * z_stride;
  const int lane = threadIdx.x % DLI_WAVE, wave = threadIdx.x / DLI_WAVE, waves = blockDim.x / DLI_WAVE;
  float s2 = 0.f, s4 = 0.f, s6 = 0.f;
  for (int i = threadIdx.x; i < ff; i += blockDim.x) {
    const float x = zr[i], x2 = x * x, x3 = x2 * x;
    s2 += x2;
    s4 += x2 * x2;
    s6 += x3 * x3;
  }
  // the three sums meet in one exchange through LDS
  s2 = wave_sum(s2); s4 = wave_sum(s4); s6 = wave_sum(s6);
  if (lane == 0) { scratch[0][wave] = s2; scratch[1][wave] = s4; scratch[2][wave] = s6; }
  __syncthreads();
  float t2 = 0.f, t4 = 0.f, t6 = 0.f;
  for (int w = 0; w < waves; ++w) { t2 += scratch[0][w]; t4 += scratch[1][w]; t6 += scratch[2][w]; }   // same order in every thread
  const float r1 = 1.f / sqrtf(t2 / (float)ff + eps), r2 = 1.f / sqrtf(t4 / (float)ff + eps), r3 = 1.f / sqrtf(t6 / (float)ff + eps);
  const float a = coef[0], b = coef[1], c = coef[2], e = coef[3];
  for (int i = threadIdx.x; i < ff; i += blockDim.x) {
    const float x = zr[i], x2 = x * x;
    const float y = a * (x * r1) + b * (x2 * r2) + c * ((x2 * x) * r3) + e;
    if (out_is_bf16) ((bf16_t*)out_)[row * out_stride + i] = (bf16_t)y;
    else ((float*)out_)[row * out_stride + i] = y;
  }
}

template <typename T>
__global__ void clamped_glu_kernel(const T* __restrict__ gate_up, int64_t stride, T* __restrict__ out, int ff, GluForm f) {
  const int64_t row = blockIdx.x;
  const int i = blockIdx.y * blockDim.x + threadIdx.x;
  if (i >= ff) return;
  const float g = to_f32(gate_up[row * stride + i]), u = to_f32(gate_up[row * stride + ff + i]);
  out[row * ff + i] = from_f32<T>(f.form == GLU_GELU ? gelu_glu(g, u) : clamped_glu(g, u, f.limit, f.alpha, f.up_shift));
}

// Eight neighbours a thread (rows and sizes of whole 16 bytes).
template <bool GELU>
__global__ __launch_bounds__(256) void clamped_glu_bf16x8_kernel(const bf16_t* __restrict__ gate_up, int64_t stride,
                                                                 bf16_t* __restrict__ out, int ff, GluForm f) {
  typedef __bf16 b8 __attribute__((ext_vector_type(8)));
  const int64_t row = blockIdx.x;
  const int i = 8 * (blockIdx.y * 256 + threadIdx.x);
  if (i >= ff) return;
  const b8 g = *reinterpret_cast<const b8*>(gate_up + row * stride + i);
  const b8 u = *reinterpret_cast<const b8*>(gate_up + row * stride + ff + i);
  b8 y;
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    if (GELU) {
      const float z = (float)g[e];
      y[e] = (bf16_t)(z * __builtin_amdgcn_rcpf(1.f + __expf(-1.5957691216057308f * (z + 0.044715f * z * z * z))) * (float)u[e]);
    } else {
      const float a = fminf((float)g[e], f.limit), b = fminf(fmaxf((float)u[e], -f.limit), f.limit);
      y[e] = (bf16_t)(a * __builtin_amdgcn_rcpf(1.f + __expf(-f.alpha * a)) * (b + f.up_shift));
    }
  }
  *reinterpret_cast<b8*>(out + row * ff + i) = y;
}

// The better of two (value, index) pairs: the larger value, the lower index on a tie.
__device__ __forceinline__ void wave_argmax(float& v, int& i) {
#pragma unroll
  for (int m = DLI_WAVE / 2; m > 0; m >>= 1) {
    const float v2 = __shfl_xor(v, m, DLI_WAVE);
    const int i2 = __shfl_xor(i, m, DLI_WAVE);
    if (v2 > v || (v2 == v && i2 < i)) { v = v2; i = i2; }
  }
}

// A wave a token. logits [rows][stride]: the first `total` columns are the router's outputs.
__global__ __launch_bounds__(64) void router_choose_kernel(const float* __restrict__ logits, int64_t stride,
                                                           const float* __restrict__ bias,
                                                           const float* __restrict__ correction, int total, int count,
                                                           int keep, int top, float scale, int sigmoid, int normalize,
                                                           int* __restrict__ ids, float* __restrict__ weights) {
  extern __shared__ float sh[];
  float *s = sh, *choice = sh + total, *gbest = sh + 2 * total;
  const int64_t row = blockIdx.x;
  const int lane = threadIdx.x;
  const float* z = logits + row * stride;
  float m = -INFINITY, sum = 0.f;
  if (sigmoid) {
    for (int i = lane; i < total; i += DLI_WAVE) s[i] = 1.f / (1.f + expf(-(z[i] + (bias != nullptr ? bias[i] : 0.f))));
    sum = 1.f;
  } else {
    for (int i = lane; i < total; i += DLI_WAVE) m = fmaxf(m, z[i] + (bias != nullptr ? bias[i] : 0.f));
    m = wave_max(m);
    for (int i = lane; i < total; i += DLI_WAVE) {
      const float e = expf(z[i] + (bias != nullptr ? bias[i] : 0.f) - m);
      s[i] = e;
      sum += e;
    }
    sum = wave_sum(sum);
  }
  for (int i = lane; i < total; i += DLI_WAVE) {
    const float p = s[i] / sum;
    s[i] = p;
    choice[i] = p + (correction != nullptr ? correction[i] : 0.f);
  }
  __syncthreads();
  if (count > 1) {
    const int per = total / count;
    for (int g = lane; g < count; g += DLI_WAVE) {
      float b = -INFINITY;
      for (int i = g * per; i < (g + 1) * per; ++i) b = fmaxf(b, choice[i]);
      gbest[g] = b;
    }
    __syncthreads();
    for (int round = 0; round < keep; ++round) {
      float bv = -INFINITY;
      int bi = 0x7fffffff;
      for (int g = lane; g < count; g += DLI_WAVE) {
        const float v = gbest[g];
        if (v == v && (v > bv || (v == bv && g < bi))) { bv = v; bi = g; }   // (NaN marks a group already kept)
      }
      wave_argmax(bv, bi);
      __syncthreads();
      if (lane == 0 && bi < count) gbest[bi] = __builtin_nanf("");
      __syncthreads();
    }
    for (int i = lane; i < total; i += DLI_WAVE) {
      const float g = gbest[i / per];
      if (g == g) choice[i] = -INFINITY;        // its group was not kept
    }
    __syncthreads();
  }
  float chosen_sum = 0.f, mine = 0.f;            // lane j keeps the j-th choice (top <= 64)
  int my_id = 0;
  for (int j = 0; j < top; ++j) {
    float bv = -INFINITY;
    int bi = 0x7fffffff;
    for (int i = lane; i < total; i += DLI_WAVE) {
      const float v = choice[i];
      if (v == v && (v > bv || (v == bv && i < bi))) { bv = v; bi = i; }      // (NaN marks an expert already chosen)
    }
    wave_argmax(bv, bi);
    bi = min(bi, total - 1);
    __syncthreads();
    const float p = s[bi];
    chosen_sum += p;
    if (lane == j) { mine = p; my_id = bi; }
    if (lane == 0) choice[bi] = __builtin_nanf("");
    __syncthreads();
  }
  if (lane < top) {
    ids[row * top + lane] = my_id;
    weights[row * top + lane] = (normalize ? mine / (chosen_sum + 1e-20f) : mine) * scale;
  }
}

#define EX_BM 32
#define EX_BN 64
#define EX_BK 16

// One workgroup. ids [slots]: the chosen expert of every (token, choice) slot; ids at or above `experts`
// (identity experts) have no rows. Leaves offsets [experts + 1], order [rows of real experts] (the slot of
// every sorted row; inside an expert's run the rows come in whatever order the counter hands out, which
// no value depends on), the tiles (expert, first sorted row) of at most tile_rows rows, and their number.
__global__ __launch_bounds__(1024) void expert_sort_kernel(const int* __restrict__ ids, int slots, int experts,
                                                           int* __restrict__ offsets, int* __restrict__ order,
                                                           int* __restrict__ tile_expert, int* __restrict__ tile_row0,
                                                           int* __restrict__ tile_count, int max_tiles, int tile_rows) {
  extern __shared__ int shi[];
  int *counts = shi, *cursor = shi + experts;
  for (int e = threadIdx.x; e < experts; e += blockDim.x) counts[e] = 0;
  __syncthreads();
  for (int i = threadIdx.x; i < slots; i += blockDim.x) {
    const int e = ids[i];
    if (e >= 0 && e < experts) atomicAdd(&counts[e], 1);
  }
  __syncthreads();
  if (threadIdx.x == 0) {
    int at = 0, tiles = 0;
    for (int e = 0; e < experts; ++e) {
      offsets[e] = at;
      cursor[e] = at;
      for (int r = 0; r < counts[e] && tiles < max_tiles; r += tile_rows) {
        tile_expert[tiles] = e;
        tile_row0[tiles] = at + r;
        ++tiles;
      }
      at += counts[e];
    }
    offsets[experts] = at;
    tile_count[0] = tiles;
  }
  __syncthreads();
  for (int i = threadIdx.x; i < slots; i += blockDim.x) {
    const int e = ids[i];
    if (e >= 0 && e < experts) order[atomicAdd(&cursor[e], 1)] = i;
  }
}

struct ExpertArgs {
  const int* tile_expert; const int* tile_row0; const int* tile_count; const int* offsets; const int* order;
  int top, width, ff;
  const float* in_weight;   // [slots], what multiplies an expert's input (nullptr: nothing)
};

// y[sorted row][ff] = clamped_glu(h[token] . w_gate[e], h[token] . w_up[e]); w_gate, w_up [experts][ff][width].
template <typename T>
__global__ __launch_bounds__(256) void expert_up_kernel(ExpertArgs p, const T* __restrict__ h, int64_t h_stride,
                                                        const T* __restrict__ w_gate, const T* __restrict__ w_up,
                                                        T* __restrict__ y, float limit, float alpha, float up_shift) {
  const int tile = blockIdx.x;
  if (tile >= p.tile_count[0]) return;
  __shared__ float as[EX_BK][EX_BM + 1], gs[EX_BK][EX_BN + 4], us[EX_BK][EX_BN + 4];
  __shared__ int tok[EX_BM];
  const int e = p.tile_expert[tile], r0 = p.tile_row0[tile], rend = p.offsets[e + 1];
  const int n0 = blockIdx.y * EX_BN;
  const int tid = threadIdx.x, tx = tid % 16, ty = tid / 16;
  if (tid < EX_BM) tok[tid] = r0 + tid < rend ? p.order[r0 + tid] / p.top : -1;
  __syncthreads();
  const T* wg = w_gate + (int64_t)e * p.ff * p.width;
  const T* wu = w_up + (int64_t)e * p.ff * p.width;
  float accg[2][4] = {}, accu[2][4] = {};
  for (int k0 = 0; k0 < p.width; k0 += EX_BK) {
    for (int i = tid; i < EX_BM * EX_BK; i += 256) {
      const int r = i / EX_BK, k = i % EX_BK;
      as[k][r] = tok[r] >= 0 && k0 + k < p.width ? to_f32(h[(int64_t)tok[r] * h_stride + k0 + k]) : 0.f;
    }
    for (int i = tid; i < EX_BN * EX_BK; i += 256) {
      const int c = i / EX_BK, k = i % EX_BK;
      const bool ok = n0 + c < p.ff && k0 + k < p.width;
      gs[k][c] = ok ? to_f32(wg[(int64_t)(n0 + c) * p.width + k0 + k]) : 0.f;
      us[k][c] = ok ? to_f32(wu[(int64_t)(n0 + c) * p.width + k0 + k]) : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < EX_BK; ++k) {
      const float a0 = as[k][ty * 2], a1 = as[k][ty * 2 + 1];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float g = gs[k][tx * 4 + j], u = us[k][tx * 4 + j];
        accg[0][j] = fmaf(a0, g, accg[0][j]);
        accg[1][j] = fmaf(a1, g, accg[1][j]);
        accu[0][j] = fmaf(a0, u, accu[0][j]);
        accu[1][j] = fmaf(a1, u, accu[1][j]);
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int r = r0 + ty * 2 + i;
    if (r >= rend) continue;
    const float iw = p.in_weight != nullptr ? p.in_weight[p.order[r]] : 1.f;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = n0 + tx * 4 + j;
      if (c < p.ff) y[(int64_t)r * p.ff + c] = from_f32<T>(clamped_glu(iw * accg[i][j], iw * accu[i][j], limit, alpha, up_shift));
    }
  }
}

// z[slot][width] = y[sorted row] . w_down[e]; w_down [experts][width][ff].
template <typename T>
__global__ __launch_bounds__(256) void expert_down_kernel(ExpertArgs p, const T* __restrict__ y, const T* __restrict__ w_down,
                                                          float* __restrict__ z) {
  const int tile = blockIdx.x;
  if (tile >= p.tile_count[0]) return;
  __shared__ float as[EX_BK][EX_BM + 1], ws[EX_BK][EX_BN + 4];
  const int e = p.tile_expert[tile], r0 = p.tile_row0[tile], rend = p.offsets[e + 1];
  const int n0 = blockIdx.y * EX_BN;
  const int tid = threadIdx.x, tx = tid % 16, ty = tid / 16;
  const T* wd = w_down + (int64_t)e * p.width * p.ff;
  float acc[2][4] = {};
  for (int k0 = 0; k0 < p.ff; k0 += EX_BK) {
    for (int i = tid; i < EX_BM * EX_BK; i += 256) {
      const int r = i / EX_BK, k = i % EX_BK;
      as[k][r] = r0 + r < rend && k0 + k < p.ff ? to_f32(y[(int64_t)(r0 + r) * p.ff + k0 + k]) : 0.f;
    }
    for (int i = tid; i < EX_BN * EX_BK; i += 256) {
      const int c = i / EX_BK, k = i % EX_BK;
      ws[k][c] = n0 + c < p.width && k0 + k < p.ff ? to_f32(wd[(int64_t)(n0 + c) * p.ff + k0 + k]) : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < EX_BK; ++k) {
      const float a0 = as[k][ty * 2], a1 = as[k][ty * 2 + 1];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float w = ws[k][tx * 4 + j];
        acc[0][j] = fmaf(a0, w, acc[0][j]);
        acc[1][j] = fmaf(a1, w, acc[1][j]);
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int r = r0 + ty * 2 + i;
    if (r >= rend) continue;
    const int64_t slot = p.order[r];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = n0 + tx * 4 + j;
      if (c < p.width) z[slot * p.width + c] = acc[i][j];
    }
  }
}

// The same two products on the matrix cores (bfloat16; width and ff multiples of 32): tiles of 16 MB sorted rows, a
// workgroup of four waves takes 64 NB features, each wave 16 NB of them for all rows of the tile.
// v_mfma_f32_16x16x32_bf16 with the weights as the first operand: lane l supplies feature l % 16 of a block and row
// l % 16 of each block of 16 rows, and the eight k values 8 (l / 16) .. + 7 of a step of 32, read straight from memory (16
// bytes a lane and operand; the rows of a tile are re-read by the four waves from the cache); the operands of the next DEPTH
// steps are on their way while a step's products are issued. A lane's results are four neighbouring features of one row.
// Every output sums its k in ascending steps of 32 whatever its tile, so a row's result depends on
// nothing beside the row. Few rows an expert (MB 1) wait for the weights alone: one block of features a wave, many steps ahead.
#define EXM_BM 64
#define EXM_FEW 16
typedef __bf16 exm_bf16x8 __attribute__((ext_vector_type(8)));
typedef float exm_float4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ exm_bf16x8 exm_load(const bf16_t* p) { return *reinterpret_cast<const exm_bf16x8*>(p); }

template <int MB, int NB, int DEPTH>
__global__ __launch_bounds__(256) void expert_up_mfma_kernel(ExpertArgs p, const bf16_t* __restrict__ h, int64_t h_stride,
                                                             const bf16_t* __restrict__ w_gate,
                                                             const bf16_t* __restrict__ w_up, bf16_t* __restrict__ y,
                                                             float limit, float alpha, float up_shift) {
  const int tile = blockIdx.x;
  if (tile >= p.tile_count[0]) return;
  const int e = p.tile_expert[tile], r0 = p.tile_row0[tile], rend = min(p.offsets[e + 1], r0 + 16 * MB);
  const int lane = threadIdx.x % DLI_WAVE, wave = threadIdx.x / DLI_WAVE;
  const int c = lane % 16, kq = (lane / 16) * 8;
  const int nw = (blockIdx.y * 4 + wave) * 16 * NB;
  const bf16_t *wg[NB], *wu[NB], *xr[MB];
#pragma unroll
  for (int nb = 0; nb < NB; ++nb) {
    const int n = min(nw + nb * 16 + c, p.ff - 1);                              // (a feature past the end repeats the last)
    wg[nb] = w_gate + ((int64_t)e * p.ff + n) * p.width + kq;
    wu[nb] = w_up + ((int64_t)e * p.ff + n) * p.width + kq;
  }
#pragma unroll
  for (int mb = 0; mb < MB; ++mb) {
    const int r = min(r0 + mb * 16 + c, rend - 1);                              // (a row past the end repeats the last)
    xr[mb] = h + (int64_t)(p.order[r] / p.top) * h_stride + kq;
  }
  exm_float4 accg[NB][MB], accu[NB][MB];
#pragma unroll
  for (int nb = 0; nb < NB; ++nb)
#pragma unroll
    for (int mb = 0; mb < MB; ++mb) accg[nb][mb] = accu[nb][mb] = exm_float4{0.f, 0.f, 0.f, 0.f};
  const int blocks = (rend - r0 + 15) / 16;                                     // blocks of 16 rows that hold a row
  exm_bf16x8 a[DEPTH][NB], b[DEPTH][NB], x[DEPTH][MB];
  auto fetch = [&](int j, int k) {
#pragma unroll
    for (int nb = 0; nb < NB; ++nb) { a[j][nb] = exm_load(wg[nb] + k); b[j][nb] = exm_load(wu[nb] + k); }
#pragma unroll
    for (int mb = 0; mb < MB; ++mb) x[j][mb] = exm_load(xr[mb] + k);             // (unconditional: clamped rows are valid memory)
  };
#pragma unroll
  for (int j = 0; j < DEPTH; ++j) fetch(j, min(32 * j, p.width - 32));
  for (int k0 = 0; k0 < p.width; k0 += 32 * DEPTH) {
#pragma unroll
    for (int j = 0; j < DEPTH; ++j) {
      const int k = k0 + 32 * j;
      exm_bf16x8 a0[NB], b0[NB], x0[MB];
#pragma unroll
      for (int nb = 0; nb < NB; ++nb) { a0[nb] = a[j][nb]; b0[nb] = b[j][nb]; }
#pragma unroll
      for (int mb = 0; mb < MB; ++mb) x0[mb] = x[j][mb];
      if (DEPTH > 1 && k >= p.width) x0[0] = exm_bf16x8{};                       // (past the last step: a product of zero)
      fetch(j, min(k + 32 * DEPTH, p.width - 32));                              // the last turn asks for its own step again
#pragma unroll
      for (int mb = 0; mb < MB; ++mb) {
        if (MB == 1 || mb < blocks) {
#pragma unroll
          for (int nb = 0; nb < NB; ++nb) {
            accg[nb][mb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a0[nb], x0[mb], accg[nb][mb], 0, 0, 0);
            accu[nb][mb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(b0[nb], x0[mb], accu[nb][mb], 0, 0, 0);
          }
        }
      }
    }
  }
#pragma unroll
  for (int mb = 0; mb < MB; ++mb) {
    const int r = r0 + mb * 16 + c;
    if (r >= rend) continue;
    const float iw = p.in_weight != nullptr ? p.in_weight[p.order[r]] : 1.f;
#pragma unroll
    for (int nb = 0; nb < NB; ++nb) {
      const int n0 = nw + nb * 16 + (lane / 16) * 4;
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (n0 + i < p.ff)
          y[(int64_t)r * p.ff + n0 + i] = (bf16_t)clamped_glu(iw * accg[nb][mb][i], iw * accu[nb][mb][i], limit, alpha, up_shift);
    }
  }
}

template <int MB, int NB, int DEPTH>
__global__ __launch_bounds__(256) void expert_down_mfma_kernel(ExpertArgs p, const bf16_t* __restrict__ y,
                                                               const bf16_t* __restrict__ w_down, float* __restrict__ z) {
  const int tile = blockIdx.x;
  if (tile >= p.tile_count[0]) return;
  const int e = p.tile_expert[tile], r0 = p.tile_row0[tile], rend = min(p.offsets[e + 1], r0 + 16 * MB);
  const int lane = threadIdx.x % DLI_WAVE, wave = threadIdx.x / DLI_WAVE;
  const int c = lane % 16, kq = (lane / 16) * 8;
  const int nw = (blockIdx.y * 4 + wave) * 16 * NB;
  const bf16_t *wd[NB], *yr[MB];
#pragma unroll
  for (int nb = 0; nb < NB; ++nb) wd[nb] = w_down + ((int64_t)e * p.width + min(nw + nb * 16 + c, p.width - 1)) * p.ff + kq;
#pragma unroll
  for (int mb = 0; mb < MB; ++mb) yr[mb] = y + (int64_t)min(r0 + mb * 16 + c, rend - 1) * p.ff + kq;
  exm_float4 acc[NB][MB];
#pragma unroll
  for (int nb = 0; nb < NB; ++nb)
#pragma unroll
    for (int mb = 0; mb < MB; ++mb) acc[nb][mb] = exm_float4{0.f, 0.f, 0.f, 0.f};
  const int blocks = (rend - r0 + 15) / 16;
  exm_bf16x8 a[DEPTH][NB], x[DEPTH][MB];
  auto fetch = [&](int j, int k) {
#pragma unroll
    for (int nb = 0; nb < NB; ++nb) a[j][nb] = exm_load(wd[nb] + k);
#pragma unroll
    for (int mb = 0; mb < MB; ++mb) x[j][mb] = exm_load(yr[mb] + k);
  };
#pragma unroll
  for (int j = 0; j < DEPTH; ++j) fetch(j, min(32 * j, p.ff - 32));
  for (int k0 = 0; k0 < p.ff; k0 += 32 * DEPTH) {
#pragma unroll
    for (int j = 0; j < DEPTH; ++j) {
      const int k = k0 + 32 * j;
      exm_bf16x8 a0[NB], x0[MB];
#pragma unroll
      for (int nb = 0; nb < NB; ++nb) a0[nb] = a[j][nb];
#pragma unroll
      for (int mb = 0; mb < MB; ++mb) x0[mb] = x[j][mb];
      if (DEPTH > 1 && k >= p.ff) x0[0] = exm_bf16x8{};
      fetch(j, min(k + 32 * DEPTH, p.ff - 32));
#pragma unroll
      for (int mb = 0; mb < MB; ++mb)
        if (MB == 1 || mb < blocks)
#pragma unroll
          for (int nb = 0; nb < NB; ++nb) acc[nb][mb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a0[nb], x0[mb], acc[nb][mb], 0, 0, 0);
    }
  }
#pragma unroll
  for (int mb = 0; mb < MB; ++mb) {
    const int r = r0 + mb * 16 + c;
    if (r >= rend) continue;
    const int64_t slot = p.order[r];
#pragma unroll
    for (int nb = 0; nb < NB; ++nb) {
      const int n0 = nw + nb * 16 + (lane / 16) * 4;
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (n0 + i < p.width) z[slot * p.width + n0 + i] = acc[nb][mb][i];
    }
  }
}

// The same two products for many rows an expert (bfloat16, sizes that are multiples of 64 and 128 as the host checks): tiles of
// EXL_BM sorted rows, a workgroup of four waves takes 128 rows of weights (the up product: 64 of each half), both
// operands through LDS 64 k at a time, the next 64 in flight in registers meanwhile. A wave takes half of the
// tile's rows and half of the weights' rows, sixteen 16 x 16 blocks. Rows in LDS are padded by 16 bytes. Every output sums its k in
// ascending steps of 32, as in the kernels above. The workgroups of one XCD take neighbouring tiles with all their
// features, so that an expert's weights are read into one L2 (or two).
#define EXL_BM 128
#define EXL_BK 64
#define EXL_LD (EXL_BK + 8)
template <bool UP>
__global__ __launch_bounds__(256, 2) void expert_tiled_kernel(ExpertArgs p, const bf16_t* __restrict__ x, int64_t x_stride,
                                                              const bf16_t* __restrict__ w0, const bf16_t* __restrict__ w1,
                                                              bf16_t* __restrict__ y, float* __restrict__ z, int blocks_n,
                                                              float limit, float alpha, float up_shift) {
  __shared__ __align__(16) bf16_t xs[2][EXL_BM * EXL_LD], ws[2][128 * EXL_LD];
  const int count = p.tile_count[0], per = (count + 7) / 8, local = blockIdx.x / 8;
  const int tile = (blockIdx.x % 8) * per + local / blocks_n, block = local % blocks_n;
  if (local / blocks_n >= per || tile >= count) return;
  const int e = p.tile_expert[tile], r0 = p.tile_row0[tile], rend = min(p.offsets[e + 1], r0 + EXL_BM);
  const int tid = threadIdx.x, lane = tid % 64, wave = __builtin_amdgcn_readfirstlane(tid / 64), c = lane % 16, g = lane / 16;
  const int wm = wave & 1, wn = wave >> 1;
  const int K = UP ? p.width : p.ff;
  // this thread's 16-byte pieces: piece tid % 8 of the rows tid / 8 + 32 m
  const bf16_t *xr[4], *wr[4];
#pragma unroll
  for (int m = 0; m < 4; ++m) {
    const int row = tid / 8 + 32 * m, r = min(r0 + row, rend - 1);              // (a row past the end repeats the last)
    xr[m] = x + (int64_t)(UP ? p.order[r] / p.top : r) * x_stride + 8 * (tid % 8);
    if (UP) wr[m] = (row < 64 ? w0 : w1) + ((int64_t)e * p.ff + 64 * block + row % 64) * K + 8 * (tid % 8);
    else wr[m] = w0 + ((int64_t)e * p.width + 128 * block + row) * K + 8 * (tid % 8);
  }
  exm_bf16x8 rx[4], rw[4];
  auto fetch = [&](int k) {
#pragma unroll
    for (int m = 0; m < 4; ++m) { rx[m] = exm_load(xr[m] + k); rw[m] = exm_load(wr[m] + k); }
  };
  auto put = [&](int buf) {
#pragma unroll
    for (int m = 0; m < 4; ++m) {
      const int at = (tid / 8 + 32 * m) * EXL_LD + 8 * (tid % 8);
      *reinterpret_cast<exm_bf16x8*>(&xs[buf][at]) = rx[m];
      *reinterpret_cast<exm_bf16x8*>(&ws[buf][at]) = rw[m];
    }
  };
  exm_float4 acc[4][4];                                                          // [weights' block][rows' block]
#pragma unroll
  for (int n = 0; n < 4; ++n)
#pragma unroll
    for (int m = 0; m < 4; ++m) acc[n][m] = exm_float4{0.f, 0.f, 0.f, 0.f};
  // the weights' blocks: gate 32 wn and 32 wn + 16, then the same of up; or 64 wn on
  int wrow[4];
#pragma unroll
  for (int n = 0; n < 4; ++n) wrow[n] = UP ? 64 * (n / 2) + 32 * wn + 16 * (n % 2) : 64 * wn + 16 * n;
  fetch(0);
  put(0);
  __syncthreads();
  int buf = 0;
  for (int k = 0; k < K; k += EXL_BK, buf ^= 1) {
    const bool more = k + EXL_BK < K;
    if (more) fetch(k + EXL_BK);
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      exm_bf16x8 a[4], b[4];
#pragma unroll
      for (int n = 0; n < 4; ++n) a[n] = exm_load(&ws[buf][(wrow[n] + c) * EXL_LD + 32 * s + 8 * g]);
#pragma unroll
      for (int m = 0; m < 4; ++m) b[m] = exm_load(&xs[buf][(64 * wm + 16 * m + c) * EXL_LD + 32 * s + 8 * g]);
#pragma unroll
      for (int n = 0; n < 4; ++n)
#pragma unroll
        for (int m = 0; m < 4; ++m) acc[n][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[n], b[m], acc[n][m], 0, 0, 0);
    }
    if (more) put(buf ^ 1);
    __syncthreads();
  }
  typedef __bf16 bf4 __attribute__((ext_vector_type(4)));
#pragma unroll
  for (int m = 0; m < 4; ++m) {
    const int r = r0 + 64 * wm + 16 * m + c;
    if (r >= rend) continue;
    if (UP) {
      const float iw = p.in_weight != nullptr ? p.in_weight[p.order[r]] : 1.f;
#pragma unroll
      for (int n = 0; n < 2; ++n) {
        bf4 o;
#pragma unroll
        for (int i = 0; i < 4; ++i) o[i] = (bf16_t)clamped_glu(iw * acc[n][m][i], iw * acc[n + 2][m][i], limit, alpha, up_shift);
        *reinterpret_cast<bf4*>(y + (int64_t)r * p.ff + 64 * block + 32 * wn + 16 * n + 4 * g) = o;
      }
    } else {
      const int64_t slot = p.order[r];
#pragma unroll
      for (int n = 0; n < 4; ++n)
        *reinterpret_cast<exm_float4*>(z + slot * p.width + 128 * block + wrow[n] + 4 * g) = acc[n][m];
    }
  }
}

// (weights nullptr: ones)
// out[token] = sum_j weights[token][j] * (ids[token][j] < experts ? z[token * top + j] : h[token])
//            + sigmoid(shared_gate[token]) * shared[token]       (the shared expert, if there is one)
template <typename T>
__global__ void expert_combine_kernel(const int* __restrict__ ids, const float* __restrict__ weights,
                                      const float* __restrict__ z, const T* __restrict__ h, int64_t h_stride,
                                      const float* __restrict__ shared_gate, int64_t gate_stride,
                                      const float* __restrict__ shared, int64_t shared_stride, float* __restrict__ out,
                                      int top, int experts, int width) {
  const int64_t row = blockIdx.x;
  const int c = blockIdx.y * blockDim.x + threadIdx.x;
  if (c >= width) return;
  float sum = 0.f;
  for (int j = 0; j < top; ++j) {
    const int e = ids[row * top + j];
    const float v = e < experts ? z[(row * top + j) * width + c] : to_f32(h[row * h_stride + c]);
    sum = fmaf(weights != nullptr ? weights[row * top + j] : 1.f, v, sum);
  }
  if (shared != nullptr) {
    const float g = shared_gate != nullptr ? 1.f / (1.f + expf(-shared_gate[row * gate_stride])) : 1.f;
    sum = fmaf(g, shared[row * shared_stride + c], sum);
  }
  out[row * width + c] = sum;
}

// The same with four columns a thread: widths, strides and addresses of whole 16-byte pieces.
template <typename T>
__global__ __launch_bounds__(256) void expert_combine4_kernel(const int* __restrict__ ids, const float* __restrict__ weights,
                                                              const float* __restrict__ z, const T* __restrict__ h, int64_t h_stride,
                                                              const float* __restrict__ shared_gate, int64_t gate_stride,
                                                              const float* __restrict__ shared, int64_t shared_stride,
                                                              float* __restrict__ out, int top, int experts, int width) {
  const int64_t row = blockIdx.x;
  const int c = (blockIdx.y * blockDim.x + threadIdx.x) * 4;
  if (c >= width) return;
  float sum[4] = {0.f, 0.f, 0.f, 0.f};
  for (int j = 0; j < top; ++j) {
    const float wt = weights != nullptr ? weights[row * top + j] : 1.f;
    float v[4];
    if (ids[row * top + j] < experts) {
      const float4 f = *reinterpret_cast<const float4*>(z + (row * top + j) * width + c);
      v[0] = f.x; v[1] = f.y; v[2] = f.z; v[3] = f.w;
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i) v[i] = to_f32(h[row * h_stride + c + i]);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) sum[i] = fmaf(wt, v[i], sum[i]);
  }
  if (shared != nullptr) {
    const float g = shared_gate != nullptr ? 1.f / (1.f + expf(-shared_gate[row * gate_stride])) : 1.f;
    const float4 f = *reinterpret_cast<const float4*>(shared + row * shared_stride + c);
    sum[0] = fmaf(g, f.x, sum[0]); sum[1] = fmaf(g, f.y, sum[1]); sum[2] = fmaf(g, f.z, sum[2]); sum[3] = fmaf(g, f.w, sum[3]);
  }
  *reinterpret_cast<float4*>(out + row * width + c) = float4{sum[0], sum[1], sum[2], sum[3]};
}

// A router that is a table: the experts of a token are the row of `table` [vocabulary][top] at its token id,
// each with the weight 1 / top. A thread a (token, choice).
__global__ void table_choose_kernel(const int* __restrict__ table, const int* __restrict__ token_ids, int n, int top,
                                    int vocab, int* __restrict__ ids, float* __restrict__ weights) {
  const int i = blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= n * top) return;
  const int t = i / top, j = i - t * top;
  const int tok = min(max(token_ids[t], 0), vocab - 1);
  ids[i] = table[(int64_t)tok * top + j];
  weights[i] = 1.f / (float)top;
}

extern "C" {

int dli_poly_norm(const float* z, int64_t z_stride, const float* coef, void* out, int64_t out_stride, int rows, int ff,
                  float eps, int out_is_bf16, hipStream_t stream) {
  if (rows <= 0) return DLI_OK;
  if (ff <= 0 || z_stride < ff || out_stride < ff) return DLI_ERR_ARGUMENT;
  poly_norm_kernel_f32in<<<rows, ff >= 4096 ? 512 : 256, 0, stream>>>(z, z_stride, coef, out, out_stride, ff, eps, out_is_bf16);
  return dli_launch_status();
}

int dli_clamped_glu(const void* gate_up, int64_t stride, void* out, int rows, int ff, int form, float limit, float alpha, float up_shift,
                    int is_bf16, hipStream_t stream) {
  if (rows <= 0) return DLI_OK;
  if (ff <= 0 || stride < 2 * (int64_t)ff || (form != GLU_CLAMPED && form != GLU_GELU)) return DLI_ERR_ARGUMENT;
  const dim3 grid(rows, (ff + 255) / 256), grid8(rows, (ff / 8 + 255) / 256);
  const GluForm f{form, limit, alpha, up_shift};
  if (is_bf16 && ff % 8 == 0 && stride % 8 == 0 && ((uintptr_t)gate_up | (uintptr_t)out) % 16 == 0) {
    if (form == GLU_GELU) clamped_glu_bf16x8_kernel<true><<<grid8, 256, 0, stream>>>((const bf16_t*)gate_up, stride, (bf16_t*)out, ff, f);
    else clamped_glu_bf16x8_kernel<false><<<grid8, 256, 0, stream>>>((const bf16_t*)gate_up, stride, (bf16_t*)out, ff, f);
  } else if (is_bf16) clamped_glu_kernel<bf16_t><<<grid, 256, 0, stream>>>((const bf16_t*)gate_up, stride, (bf16_t*)out, ff, f);
  else clamped_glu_kernel<float><<<grid, 256, 0, stream>>>((const float*)gate_up, stride, (float*)out, ff, f);
  return dli_launch_status();
}

int dli_router_choose(const float* logits, int64_t stride, const float* bias, const float* correction, int rows, int total, int count, int keep,
                      int top, float scale, int sigmoid, int normalize, int* ids, float* weights, hipStream_t stream) {
  if (rows <= 0) return DLI_OK;
  if (total <= 0 || total > 4096 || stride < total || top < 1 || top > 64 || top > total || count < 1 || total % count ||
      keep < 1 || keep > count || (int64_t)keep * (total / count) < top)
    return DLI_ERR_ARGUMENT;
  router_choose_kernel<<<rows, 64, (2 * total + count) * sizeof(float), stream>>>(logits, stride, bias, correction, total, count, keep,
                                                                                  top, scale, sigmoid, normalize, ids, weights);
  return dli_launch_status();
}

// Whether the matrix-core kernels take these sizes, and the rows of a tile of the kernels that will run.
static bool expert_mfma(int width, int ff, int is_bf16) { return is_bf16 && width % 32 == 0 && ff % 32 == 0; }
// Many rows an expert, and sizes that tile: the kernels that pass both operands through LDS.
static bool expert_tiled(int64_t slots, int experts, int width, int ff, int is_bf16) {
  return is_bf16 && width % 128 == 0 && ff % 64 == 0 && slots >= 48 * (int64_t)experts;
}
// Few rows an expert: the kernels that wait for the weights alone.
static bool expert_few(int64_t slots, int experts) { return slots <= 16 * (int64_t)experts; }
int dli_expert_tile_rows(int64_t slots, int experts, int width, int ff, int is_bf16) {
  if (expert_tiled(slots, experts, width, ff, is_bf16)) return EXL_BM;
  if (!expert_mfma(width, ff, is_bf16)) return EX_BM;
  return expert_few(slots, experts) ? EXM_FEW : EXM_BM;
}

// The experts' part of a mixture for `rows` tokens: sort, up product with activation, down product.
// ids [rows][top]; scratch: offsets [experts + 1], order [rows * top], tile_expert and tile_row0 [max_tiles],
// tile_count [1] (int32), y [rows * top][ff] (T), z [rows * top][width] (float32). in_weight [rows][top] (may be nullptr):
// what each slot's expert input is multiplied by.
int dli_expert_products(const int* ids, const void* h, int64_t h_stride, const void* w_gate, const void* w_up,
                        const void* w_down, int* offsets, int* order, int* tile_expert, int* tile_row0, int* tile_count,
                        int max_tiles, void* y, float* z, const float* in_weight, int rows, int top, int experts, int width,
                        int ff, float limit, float alpha, float up_shift, int is_bf16, hipStream_t stream) {
  if (rows <= 0) return DLI_OK;
  const int64_t slots = (int64_t)rows * top;
  if (top < 1 || experts < 1 || experts > 4096 || width <= 0 || ff <= 0 || h_stride < width || slots > (1 << 30) ||
      max_tiles < 1 || max_tiles > 65535 * 16)
    return DLI_ERR_ARGUMENT;
  const bool mfma = expert_mfma(width, ff, is_bf16);
  if (mfma && ((h_stride % 8) || ((uintptr_t)h % 16) || ((uintptr_t)w_gate % 16) || ((uintptr_t)w_up % 16) ||
               ((uintptr_t)w_down % 16) || ((uintptr_t)y % 16)))
    return DLI_ERR_ARGUMENT;
  expert_sort_kernel<<<1, 1024, 2 * experts * sizeof(int), stream>>>(ids, (int)slots, experts, offsets, order, tile_expert,
                                                                     tile_row0, tile_count, max_tiles,
                                                                     dli_expert_tile_rows(slots, experts, width, ff, is_bf16));
  if (dli_launch_status() != DLI_OK) return DLI_ERR_LAUNCH;
  ExpertArgs p;
  p.tile_expert = tile_expert; p.tile_row0 = tile_row0; p.tile_count = tile_count; p.offsets = offsets; p.order = order;
  p.top = top; p.width = width; p.ff = ff; p.in_weight = in_weight;
  if (expert_tiled(slots, experts, width, ff, is_bf16)) {
    const unsigned tiles8 = 8 * ((max_tiles + 7) / 8);
    if ((int64_t)tiles8 * (ff / 64 + width / 128) > 0x7fffffff || ((uintptr_t)z % 16)) return DLI_ERR_ARGUMENT;
    expert_tiled_kernel<true><<<tiles8 * (ff / 64), 256, 0, stream>>>(p, (const bf16_t*)h, h_stride, (const bf16_t*)w_gate,
                                                                      (const bf16_t*)w_up, (bf16_t*)y, nullptr, ff / 64, limit, alpha, up_shift);
    expert_tiled_kernel<false><<<tiles8 * (width / 128), 256, 0, stream>>>(p, (const bf16_t*)y, ff, (const bf16_t*)w_down, nullptr,
                                                                           nullptr, z, width / 128, 0.f, 0.f, 0.f);
    return dli_launch_status();
  }
  const int bn = !mfma ? EX_BN : expert_few(slots, experts) ? 64 : 128;
  const dim3 up_grid(max_tiles, (ff + bn - 1) / bn), down_grid(max_tiles, (width + bn - 1) / bn);
#define EXM_LAUNCH(MB, NB, DU, DD)                                                                                                 \
  expert_up_mfma_kernel<MB, NB, DU><<<up_grid, 256, 0, stream>>>(p, (const bf16_t*)h, h_stride, (const bf16_t*)w_gate,             \
                                                                 (const bf16_t*)w_up, (bf16_t*)y, limit, alpha, up_shift);          \
  expert_down_mfma_kernel<MB, NB, DD><<<down_grid, 256, 0, stream>>>(p, (const bf16_t*)y, (const bf16_t*)w_down, z)
  if (mfma && expert_few(slots, experts)) {
    EXM_LAUNCH(1, 1, 8, 8);
  } else if (mfma) {
    EXM_LAUNCH(4, 2, 1, 1);
  } else if (is_bf16) {
    expert_up_kernel<bf16_t><<<up_grid, 256, 0, stream>>>(p, (const bf16_t*)h, h_stride, (const bf16_t*)w_gate,
                                                          (const bf16_t*)w_up, (bf16_t*)y, limit, alpha, up_shift);
    expert_down_kernel<bf16_t><<<down_grid, 256, 0, stream>>>(p, (const bf16_t*)y, (const bf16_t*)w_down, z);
  } else {
    expert_up_kernel<float><<<up_grid, 256, 0, stream>>>(p, (const float*)h, h_stride, (const float*)w_gate,
                                                         (const float*)w_up, (float*)y, limit, alpha, up_shift);
    expert_down_kernel<float><<<down_grid, 256, 0, stream>>>(p, (const float*)y, (const float*)w_down, z);
  }
  return dli_launch_status();
}

int dli_expert_combine(const int* ids, const float* weights, const float* z, const void* h, int64_t h_stride,
                       const float* shared_gate, int64_t gate_stride, const float* shared, int64_t shared_stride, float* out,
                       int rows, int top, int experts, int width, int is_bf16, hipStream_t stream) {
  if (rows <= 0) return DLI_OK;
  if (top < 1 || width <= 0 || h_stride < width || (shared != nullptr && shared_stride < width)) return DLI_ERR_ARGUMENT;
  auto whole = [](const void* at) { return (uintptr_t)at % 16 == 0; };
  // (with few rows the extra workgroups of one column a thread hide more of the wait)
  const bool fours = rows >= 256 && width % 4 == 0 && whole(z) && whole(out) && (shared == nullptr || (whole(shared) && shared_stride % 4 == 0));
  const int cols = fours ? 1024 : 256;
  const dim3 grid(rows, (width + cols - 1) / cols);
#define COMBINE(KERNEL, T) KERNEL<T><<<grid, 256, 0, stream>>>(ids, weights, z, (const T*)h, h_stride, shared_gate, gate_stride, \
                                                               shared, shared_stride, out, top, experts, width)
  if (is_bf16) { if (fours) COMBINE(expert_combine4_kernel, bf16_t); else COMBINE(expert_combine_kernel, bf16_t); }
  else { if (fours) COMBINE(expert_combine4_kernel, float); else COMBINE(expert_combine_kernel, float); }
#undef COMBINE
  return dli_launch_status();
}

int dli_table_choose(const int* table, const int* token_ids, int n, int top, int vocab, int* ids, float* weights,
                     hipStream_t stream) {
  if (n <= 0) return DLI_OK;
  if (top <= 0 || vocab <= 0 || (int64_t)n * top > 0x7fffffff) return DLI_ERR_ARGUMENT;
  table_choose_kernel<<<(n * top + 255) / 256, 256, 0, stream>>>(table, token_ids, n, top, vocab, ids, weights);
  return dli_launch_status();
}

}  // extern "C"
