// The recurrence under step sizes of csrc/scalar_gate_scan.hip for the portions of a bfloat16 step, on the bfloat16
// matrix cores and without a chain over the tokens. Per head, with dt_t = softplus(step_t + bias) and A_t the running sum of
// -exp(rate) dt_t (never above zero):
//
//   S_t = exp(A_t - A_(t-1)) S_(t-1) + dt_t k_t v_t^T,   o_t = S_t^T q_t + skip v_t,
//
// where q and k (N values) belong to a group of heads and v (V values) to a head; all three are bfloat16 numbers, the step
// sizes, decays and the state are 32-bit. An entry's rows are cut into tiles of 256 tokens:
//
//   tile state   what a tile adds to the state by its end, sum_t w_t k_t v_t^T with w_t = exp(A_end - A_t) dt_t, and exp(A_end).
//                w_t v_t goes into the product as the sum of three bfloat16 numbers (24 bits: itself), sums in 32-bit
//   carry        a thread an element walks an entry's tiles: the state in 32-bit from the request's slot (zeros where the
//                entry begins at position 0) to the slot; the state at each tile's beginning is left as the sum of two
//                bfloat16 numbers (an operand of the results alone; what is carried on is never rounded)
//   tile result  o_t = exp(A_t) S_in^T q_t + sum_(s <= t in the tile) (q_t . k_s) exp(A_t - A_s) dt_s v_s + skip v_t; the scores
//                are products of bfloat16 numbers summed in 32-bit, and go into the second product as two bfloat16 numbers
//
// All products run on v_mfma_f32_16x16x32_bf16. Results are made in transposed form (K Q^T, then V^T P^T), so a lane holds scores of
// ONE token: of the tokens 4 g + i and 16 + 4 g + i (g = lane / 16, i < 4) of a run of 32, which are the eight k of the
// second product as they stand; its other operand, and both of the tile state's, come out of rows in LDS by the
// transposing read (ds_read_b64_tr_b16: sixteen lanes read four rows of sixteen, each gets a column of four).
//
// A_t is summed in double and kept as two floats, high and low: a difference is then good to its own last bit, where a
// running sum in the hundreds as one float would be good to 1e-5.
#include "common.h"

typedef __bf16 ss_bf8 __attribute__((ext_vector_type(8)));
typedef __bf16 ss_bf4 __attribute__((ext_vector_type(4)));
typedef float ss_f4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) ss_bf4* ss_lds4;

#define SS_TILE 256

template <int I> struct SsInt { static constexpr int value = I; };

struct SsArgs {
  const bf16_t* q; const bf16_t* k; const bf16_t* v; int64_t stride;   // [rows][stride], each at its first column
  const float* step; int64_t step_stride; const float* bias; const float* rate; const float* skip;
  float* state; int64_t state_stride;                                  // [heads][V][N] a slot
  const int* q_start; const int* positions; const int* state_slots;
  const int* tile_entry; const int* tile_q0;
  float* ends;                     // [tiles][heads][V][N]
  float* total;                    // [tiles][heads]
  bf16_t* in_hi; bf16_t* in_lo;    // [tiles][heads][V][N]
  float* o; int64_t o_stride;
  int heads, qk_heads, V, N;
};

// This thread's token (of 256): its step size, and the running sum of the logarithms (base 2) of the decays up to it; `all`: the
// whole tile's. sh: four doubles.
__device__ __forceinline__ void ss_steps(const SsArgs& p, int row0, int n_rows, int head, double* sh, float* dt, double* run, double* all) {
  const int t = threadIdx.x, lane = t % 64, wave = t / 64;
  const float x = p.step[(int64_t)(row0 + min(t, n_rows - 1)) * p.step_stride + head] + p.bias[head];
  *dt = t < n_rows ? fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))) : 0.f;
  double la = (double)(*dt * -expf(p.rate[head])) * 1.4426950408889634;
#pragma unroll
  for (int d = 1; d < 64; d <<= 1) {
    const double up = __shfl_up(la, d, DLI_WAVE);
    if (lane >= d) la += up;
  }
  if (lane == 63) sh[wave] = la;
  __syncthreads();
  double before = 0.0, sum = 0.0;
#pragma unroll
  for (int w = 0; w < 4; ++w) {
    if (w < wave) before += sh[w];
    sum += sh[w];
  }
  *run = before + la;
  *all = sum;
}

__device__ __forceinline__ ss_bf8 ss_column(const bf16_t* at, int row_stride) {
  const ss_bf4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((ss_lds4)at);
  const ss_bf4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((ss_lds4)(at + 16 * row_stride));
  return __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
}

// N = 32 NT. A workgroup a (tile, head, 64 values); a wave makes 16 of every 64 keys' rows of the tile's state.
template <int NT>
__global__ __launch_bounds__(256, 2) void state_space_tile_state_kernel(SsArgs p) {
  constexpr int N = 32 * NT, LK = N + 8, LV = 64 + 8, KP = NT, NB = (NT + 1) / 2;   // KP: 16-byte pieces of k a thread brings
  __shared__ __align__(16) bf16_t sk[64 * LK], sv[3][64 * LV];
  __shared__ float sw[SS_TILE];
  __shared__ double sh[4];
  const int tid = threadIdx.x, lane = tid % 64, wave = __builtin_amdgcn_readfirstlane(tid / 64), col = lane & 15, grp = lane >> 4;
  const int tile = blockIdx.x, head = blockIdx.y, v0 = blockIdx.z * 64;
  const int entry = p.tile_entry[tile], q0 = p.tile_q0[tile];
  const int row0 = p.q_start[entry] + q0, n_rows = min(SS_TILE, p.q_start[entry + 1] - row0);
  if (n_rows <= 0) return;
  const bf16_t* kk = p.k + (int64_t)(head / (p.heads / p.qk_heads)) * N;
  const bf16_t* vv = p.v + (int64_t)head * p.V + v0;
  const int vlast = min(64, p.V - v0) - 8;                  // (V a multiple of 8)
  ss_bf8 rk[KP], rv[2];
  auto fetch = [&](int c0) {                                // rows past the last: the last again, with a weight of zero
#pragma unroll
    for (int m = 0; m < KP; ++m) {
      const int idx = tid + 256 * m, t = idx / (4 * NT), c = idx % (4 * NT);
      rk[m] = *reinterpret_cast<const ss_bf8*>(kk + (int64_t)(row0 + min(c0 + t, n_rows - 1)) * p.stride + 8 * c);
    }
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      const int idx = tid + 256 * m, t = idx / 8, c = idx % 8;
      rv[m] = *reinterpret_cast<const ss_bf8*>(vv + (int64_t)(row0 + min(c0 + t, n_rows - 1)) * p.stride + min(8 * c, vlast));
    }
  };
  fetch(0);
  {
    float dt;
    double run, all;
    ss_steps(p, row0, n_rows, head, sh, &dt, &run, &all);
    sw[tid] = __builtin_amdgcn_exp2f((float)(all - run)) * dt;
    if (tid == 0 && v0 == 0) p.total[(int64_t)tile * p.heads + head] = __builtin_amdgcn_exp2f((float)all);
  }
  ss_f4 acc[NB][4];
#pragma unroll
  for (int n = 0; n < NB; ++n)
#pragma unroll
    for (int v = 0; v < 4; ++v) acc[n][v] = ss_f4{0.f, 0.f, 0.f, 0.f};
  for (int c0 = 0; c0 < n_rows; c0 += 64) {
    __syncthreads();
#pragma unroll
    for (int m = 0; m < KP; ++m) {
      const int idx = tid + 256 * m, t = idx / (4 * NT), c = idx % (4 * NT);
      *reinterpret_cast<ss_bf8*>(&sk[t * LK + 8 * c]) = rk[m];
    }
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      const int idx = tid + 256 * m, t = idx / 8, c = idx % 8;
      const float w = sw[c0 + t];
      ss_bf8 h[3];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float x = w * (float)rv[m][e];
        h[0][e] = (bf16_t)x;
        const float r = x - (float)h[0][e];
        h[1][e] = (bf16_t)r;
        h[2][e] = (bf16_t)(r - (float)h[1][e]);
      }
#pragma unroll
      for (int j = 0; j < 3; ++j) *reinterpret_cast<ss_bf8*>(&sv[j][t * LV + 8 * c]) = h[j];
    }
    __syncthreads();
    if (c0 + 64 < n_rows) fetch(c0 + 64);
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      const int at = 32 * s + 4 * grp + col / 4;
      ss_bf8 kf[NB];
#pragma unroll
      for (int n = 0; n < NB; ++n) kf[n] = ss_column(&sk[at * LK + min(16 * (wave + 4 * n), N - 16) + 4 * (col % 4)], LK);
#pragma unroll
      for (int v = 0; v < 4; ++v)
#pragma unroll
        for (int j = 0; j < 3; ++j) {
          const ss_bf8 vf = ss_column(&sv[j][at * LV + 16 * v + 4 * (col % 4)], LV);
#pragma unroll
          for (int n = 0; n < NB; ++n) acc[n][v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[n], vf, acc[n][v], 0, 0, 0);
        }
    }
  }
  float* out = p.ends + ((int64_t)tile * p.heads + head) * p.V * N;
#pragma unroll
  for (int n = 0; n < NB; ++n) {
    const int nb = 16 * (wave + 4 * n);
    if (nb >= N) continue;
#pragma unroll
    for (int v = 0; v < 4; ++v) {                           // acc[n][v][i]: key nb + 4 grp + i, value 16 v + col
      const int vi = v0 + 16 * v + col;
      if (vi < p.V) *reinterpret_cast<ss_f4*>(out + (int64_t)vi * N + nb + 4 * grp) = acc[n][v];
    }
  }
}

// Two neighbours of the state a thread, of the entry that a tile with tile_q0 0 begins. (The tile is the grid's slowest
// coordinate: the workgroups of such tiles, which do all the work, then lie side by side and go round all XCDs.)
__global__ __launch_bounds__(256) void state_space_carry_kernel(SsArgs p) {
  typedef float f2 __attribute__((ext_vector_type(2)));
  typedef __bf16 b2 __attribute__((ext_vector_type(2)));
  constexpr int AHEAD = 8;                                  // tiles asked for at once, the next ones before these are walked
  const int first = blockIdx.z, head = blockIdx.y, i = 2 * (blockIdx.x * 256 + threadIdx.x), size = p.V * p.N;
  if (p.tile_q0[first] != 0 || i >= size) return;
  const int entry = p.tile_entry[first];
  const int row0 = p.q_start[entry], tiles = (p.q_start[entry + 1] - row0 + SS_TILE - 1) / SS_TILE;
  float* st = p.state + (int64_t)p.state_slots[entry] * p.state_stride + (int64_t)head * size + i;
  const int64_t hop = (int64_t)p.heads * size;
  const int64_t at = ((int64_t)first * p.heads + head) * size + i;
  f2 S = *reinterpret_cast<const f2*>(st);
  if (p.positions[row0] == 0) S = f2{0.f, 0.f};
  f2 e[2][AHEAD];
  float a[2][AHEAD];
  auto fetch = [&](int w, int t0) {
#pragma unroll
    for (int j = 0; j < AHEAD; ++j) {                       // (tiles past the last repeat it)
      const int t = min(t0 + j, tiles - 1);
      e[w][j] = *reinterpret_cast<const f2*>(p.ends + at + t * hop);
      a[w][j] = p.total[(int64_t)(first + t) * p.heads + head];
    }
  };
  auto walk = [&](int w, int t0) {
#pragma unroll
    for (int j = 0; j < AHEAD; ++j)
      if (t0 + j < tiles) {
        b2 hi, lo;
#pragma unroll
        for (int c = 0; c < 2; ++c) {
          hi[c] = (bf16_t)S[c];
          lo[c] = (bf16_t)(S[c] - (float)hi[c]);
          S[c] = fmaf(a[w][j], S[c], e[w][j][c]);
        }
        *reinterpret_cast<b2*>(p.in_hi + at + (t0 + j) * hop) = hi;
        *reinterpret_cast<b2*>(p.in_lo + at + (t0 + j) * hop) = lo;
      }
  };
  fetch(0, 0);
  for (int t0 = 0; t0 < tiles; t0 += 2 * AHEAD) {
    if (t0 + AHEAD < tiles) fetch(1, t0 + AHEAD);
    walk(0, t0);
    if (t0 + AHEAD >= tiles) break;
    if (t0 + 2 * AHEAD < tiles) fetch(0, t0 + 2 * AHEAD);
    walk(1, t0 + AHEAD);
  }
  *reinterpret_cast<f2*>(st) = S;
}

// A workgroup a (tile, head, 64 values, half of the tile's runs of 16 tokens). Of the sixteen runs wave w takes j = 2 w + half
// and 15 - j, so that all waves see as many earlier tokens. What is multiplied passes through LDS 64 rows at a time, the
// next in flight meanwhile: first the two halves of the state at the tile's beginning (64 values' rows of N), then k and v of
// 64 tokens after the other.
template <int NT>
__global__ __launch_bounds__(256, 2) void state_space_tile_result_kernel(SsArgs p) {
  constexpr int N = 32 * NT, LK = N + 8, LV = 64 + 8, KP = NT;
  __shared__ __align__(16) bf16_t sk[64 * LK], sv[64 * LV];
  __shared__ __align__(16) float s_hi[SS_TILE], s_lo[SS_TILE], s_dt[SS_TILE];
  __shared__ double sh[4];
  const int tid = threadIdx.x, lane = tid % 64, wave = __builtin_amdgcn_readfirstlane(tid / 64), col = lane & 15, grp = lane >> 4;
  const int tile = blockIdx.x, head = blockIdx.y, v0 = (blockIdx.z >> 1) * 64;
  const int entry = p.tile_entry[tile], q0 = p.tile_q0[tile];
  const int start = p.q_start[entry], row0 = start + q0, n_rows = min(SS_TILE, p.q_start[entry + 1] - row0);
  if (n_rows <= 0) return;
  const int half = 2 * wave + (blockIdx.z & 1);
  const int run[2] = {16 * half, 16 * (15 - half)};         // the first token of each of this wave's runs
  const int blocks = (n_rows + 63) / 64;
  const int group = head / (p.heads / p.qk_heads);
  const bf16_t* qq = p.q + (int64_t)group * N;
  const bf16_t* kk = p.k + (int64_t)group * N;
  const bf16_t* vv = p.v + (int64_t)head * p.V + v0;
  const int vlast = min(64, p.V - v0) - 8;
  const int64_t in_at = ((int64_t)tile * p.heads + head) * p.V * N;
  const bool carried = q0 != 0 || p.positions[start] != 0;  // (else the state at the tile's beginning is zero)
  ss_bf8 rk[KP], rv[2];
  auto fetch = [&](int stage) {                             // (rows past the last: the last again; such tokens have a step of zero)
    const bf16_t* base = stage == -2 ? p.in_hi + in_at : stage == -1 ? p.in_lo + in_at : kk + (int64_t)row0 * p.stride;
    const int64_t hop = stage < 0 ? N : p.stride;
    const int r0 = stage < 0 ? v0 : 64 * stage, last = stage < 0 ? p.V - 1 : n_rows - 1;
#pragma unroll
    for (int m = 0; m < KP; ++m) {
      const int idx = tid + 256 * m, t = idx / (4 * NT), c = idx % (4 * NT);
      rk[m] = *reinterpret_cast<const ss_bf8*>(base + min(r0 + t, last) * hop + 8 * c);
    }
    if (stage >= 0)
#pragma unroll
      for (int m = 0; m < 2; ++m) {
        const int idx = tid + 256 * m, t = idx / 8, c = idx % 8;
        rv[m] = *reinterpret_cast<const ss_bf8*>(vv + (int64_t)(row0 + min(64 * stage + t, n_rows - 1)) * p.stride + min(8 * c, vlast));
      }
  };
  const int first = carried ? -2 : 0;
  fetch(first);
  ss_bf8 qb[2][NT];
#pragma unroll
  for (int b = 0; b < 2; ++b) {
    const bf16_t* qr = qq + (int64_t)(row0 + min(run[b] + col, n_rows - 1)) * p.stride + 8 * grp;
#pragma unroll
    for (int d = 0; d < NT; ++d) qb[b][d] = *reinterpret_cast<const ss_bf8*>(qr + 32 * d);
  }
  {
    float dt;
    double sum, all;
    ss_steps(p, row0, n_rows, head, sh, &dt, &sum, &all);
    s_hi[tid] = (float)sum;
    s_lo[tid] = (float)(sum - (double)(float)sum);
    s_dt[tid] = dt;
  }
  ss_f4 acc[2][4];
#pragma unroll
  for (int b = 0; b < 2; ++b)
#pragma unroll
    for (int v = 0; v < 4; ++v) acc[b][v] = ss_f4{0.f, 0.f, 0.f, 0.f};
  float t_hi[2], t_lo[2];
  for (int stage = first; stage < blocks; ++stage) {
    __syncthreads();                                        // the stage before has been read
#pragma unroll
    for (int m = 0; m < KP; ++m) {
      const int idx = tid + 256 * m, t = idx / (4 * NT), c = idx % (4 * NT);
      *reinterpret_cast<ss_bf8*>(&sk[t * LK + 8 * c]) = rk[m];
    }
    if (stage >= 0)
#pragma unroll
      for (int m = 0; m < 2; ++m) {
        const int idx = tid + 256 * m, t = idx / 8, c = idx % 8;
        *reinterpret_cast<ss_bf8*>(&sv[t * LV + 8 * c]) = rv[m];
      }
    __syncthreads();
    if (stage + 1 < blocks) fetch(stage + 1);
    if (stage < 0) {
#pragma unroll
      for (int v = 0; v < 4; ++v)
#pragma unroll
        for (int d = 0; d < NT; ++d) {
          const ss_bf8 f = *reinterpret_cast<const ss_bf8*>(&sk[(16 * v + col) * LK + 32 * d + 8 * grp]);
#pragma unroll
          for (int b = 0; b < 2; ++b) acc[b][v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f, qb[b][d], acc[b][v], 0, 0, 0);
        }
      if (stage == -1)
#pragma unroll
        for (int b = 0; b < 2; ++b) {
          const float f = __builtin_amdgcn_exp2f(s_hi[run[b] + col] + s_lo[run[b] + col]);
#pragma unroll
          for (int v = 0; v < 4; ++v) acc[b][v] *= f;
        }
      continue;
    }
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      t_hi[b] = s_hi[run[b] + col];
      t_lo[b] = s_lo[run[b] + col];
    }
    // 32 tokens from j0 on against the wave's runs from FROM on
    auto against = [&](auto from, int k) {
      constexpr int FROM = decltype(from)::value;
      const int j0 = 64 * stage + 32 * k;
      ss_f4 s[2][2];
#pragma unroll
      for (int b = FROM; b < 2; ++b) s[b][0] = s[b][1] = ss_f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int d = 0; d < NT; ++d) {
          const ss_bf8 kf = *reinterpret_cast<const ss_bf8*>(&sk[(32 * k + 16 * u + col) * LK + 32 * d + 8 * grp]);
#pragma unroll
          for (int b = FROM; b < 2; ++b) s[b][u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qb[b][d], s[b][u], 0, 0, 0);
        }
      // s[b][u][i]: token j0 + 16 u + 4 grp + i against this lane's token of run b
      ss_bf8 ph[2], pl[2];
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        const int at = j0 + 16 * u + 4 * grp;
        const ss_f4 hi = *reinterpret_cast<const ss_f4*>(&s_hi[at]), lo = *reinterpret_cast<const ss_f4*>(&s_lo[at]);
        const ss_f4 dt = *reinterpret_cast<const ss_f4*>(&s_dt[at]);
#pragma unroll
        for (int b = FROM; b < 2; ++b)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const float x = (t_hi[b] - hi[i]) + (t_lo[b] - lo[i]);
            const float w = s[b][u][i] * (__builtin_amdgcn_exp2f(at + i <= run[b] + col ? x : -INFINITY) * dt[i]);
            const bf16_t h = (bf16_t)w;
            ph[b][4 * u + i] = h;
            pl[b][4 * u + i] = (bf16_t)(w - (float)h);
          }
      }
#pragma unroll
      for (int v = 0; v < 4; ++v) {
        const ss_bf8 vf = ss_column(&sv[(32 * k + 4 * grp + col / 4) * LV + 16 * v + 4 * (col % 4)], LV);
#pragma unroll
        for (int b = FROM; b < 2; ++b) {
          acc[b][v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, ph[b], acc[b][v], 0, 0, 0);
          acc[b][v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pl[b], acc[b][v], 0, 0, 0);
        }
      }
    };
#pragma unroll 1
    for (int k = 0; k < 2; ++k) {
      const int j0 = 64 * stage + 32 * k;                   // (the second run lies behind the first)
      if (j0 <= run[0] + 15) against(SsInt<0>{}, k);
      else if (j0 <= run[1] + 15 && run[1] < n_rows) against(SsInt<1>{}, k);
    }
  }
  const float skip = p.skip != nullptr ? p.skip[head] : 0.f;
#pragma unroll
  for (int b = 0; b < 2; ++b) {
    const int t = run[b] + col;
    if (t >= n_rows) continue;
    const bf16_t* vr = vv + (int64_t)(row0 + t) * p.stride;
    float* out = p.o + (int64_t)(row0 + t) * p.o_stride + (int64_t)head * p.V + v0;
#pragma unroll
    for (int v = 0; v < 4; ++v) {                           // acc[b][v][i]: value 16 v + 4 grp + i of token t
      const int c = 16 * v + 4 * grp;
      if (v0 + c >= p.V) continue;
      const ss_bf4 x = *reinterpret_cast<const ss_bf4*>(vr + c);
      ss_f4 y;
#pragma unroll
      for (int i = 0; i < 4; ++i) y[i] = fmaf(skip, (float)x[i], acc[b][v][i]);
      *reinterpret_cast<ss_f4*>(out + c) = y;
    }
  }
}

extern "C" {

int dli_state_space_tile_rows() { return SS_TILE; }

int dli_state_space_tiles_supports(int state_size, int value_dim) {
  return state_size > 0 && state_size % 32 == 0 && state_size <= 128 && value_dim > 0 && value_dim % 8 == 0;
}

// q, k, v: bfloat16 columns of one matrix of row stride `stride`. Tiles of dli_state_space_tile_rows() rows, of each entry all of
// them, by entry and then by row. Scratch: ends [tiles][heads][V][N] and total [tiles][heads] float, in_hi and in_lo
// [tiles][heads][V][N] bfloat16.
int dli_state_space_tiles(const void* q, const void* k, const void* v, int64_t stride, const float* step, int64_t step_stride,
                          const float* bias, const float* rate, const float* skip, float* state, int64_t state_stride,
                          const int* q_start, const int* positions, const int* state_slots, const int* tile_entry,
                          const int* tile_q0, int tiles, float* ends, float* total, void* in_hi, void* in_lo, float* o,
                          int64_t o_stride, int heads, int qk_heads, int state_size, int value_dim, hipStream_t stream) {
  if (tiles <= 0) return DLI_OK;
  const int64_t size = (int64_t)state_size * value_dim;
  if (!dli_state_space_tiles_supports(state_size, value_dim) || heads <= 0 || heads > 65535 || qk_heads <= 0 || heads % qk_heads ||
      stride % 8 || o_stride % 4 || o_stride < (int64_t)heads * value_dim || step_stride < heads || state_stride < heads * size ||
      state_stride % 4 || ((uintptr_t)q | (uintptr_t)k | (uintptr_t)v | (uintptr_t)state | (uintptr_t)ends | (uintptr_t)in_hi |
                           (uintptr_t)in_lo | (uintptr_t)o) % 16)
    return DLI_ERR_ARGUMENT;
  SsArgs p;
  p.q = (const bf16_t*)q; p.k = (const bf16_t*)k; p.v = (const bf16_t*)v; p.stride = stride; p.step = step;
  p.step_stride = step_stride; p.bias = bias; p.rate = rate; p.skip = skip; p.state = state; p.state_stride = state_stride;
  p.q_start = q_start; p.positions = positions; p.state_slots = state_slots; p.tile_entry = tile_entry; p.tile_q0 = tile_q0;
  p.ends = ends; p.total = total; p.in_hi = (bf16_t*)in_hi; p.in_lo = (bf16_t*)in_lo; p.o = o; p.o_stride = o_stride;
  p.heads = heads; p.qk_heads = qk_heads; p.V = value_dim; p.N = state_size;
  const dim3 grid(tiles, heads, (value_dim + 63) / 64), result(tiles, heads, 2 * grid.z), carry((unsigned)((size / 2 + 255) / 256), heads, tiles);
  if (result.z > 65535 || carry.z > 65535) return DLI_ERR_ARGUMENT;
#define SS_CASE(NT)                                                                  \
  case NT:                                                                           \
    state_space_tile_state_kernel<NT><<<grid, 256, 0, stream>>>(p);                  \
    state_space_carry_kernel<<<carry, 256, 0, stream>>>(p);                          \
    state_space_tile_result_kernel<NT><<<result, 256, 0, stream>>>(p);                 \
    break;
  switch (state_size / 32) { SS_CASE(1) SS_CASE(2) SS_CASE(3) SS_CASE(4) }
#undef SS_CASE
  return dli_launch_status();
}

}  // extern "C"
