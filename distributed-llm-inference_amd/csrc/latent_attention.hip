// Attention through a latent: what is cached per token is one normalised vector c of `rank` values, from
// which every head's keys and values are linear maps, k_h = U_h c and v_h = W_h c. The scores of head h are
// then (U_h^T q_h) . c and its result W_h (sum_j p_j c_j): the attention itself runs over the cached
// vectors as one shared kv head whose values are its keys, between two small products per head.
//
//   latent_norm_cache  from a step's 32-bit projections: the query's latent and the kv latent each
//                      divided by their root mean square and multiplied by a weight; the first goes out
//                      in T (the operand of the queries' product), the second into the token's cache
//                      slot, as a key (page [slot][rank + rot]) and, if there are value pages, as a value
//                      (page [rank][slot]). rot > 0: the rot columns behind the latent are one key part shared
//                      by all heads, rotated (component i with i + rot/2) and written behind the latent.
//                      rank 0: the query's latent alone (a layer that reads another's latents)
//   head_products      out[t][h] = M_h x[t][h] for every head, M [heads][m][k], a head's x and out lying in
//                      rows of a given length (so that a part of each can be read or written); optionally
//                      multiplied by sigmoid(gate), element by element or one number a head. The same launch
//                      can rotate rot components that lie behind a head's x into the place behind its out.
//                      On the matrix cores for bfloat16 and k, strides of whole 16 bytes; else on the vector
//                      units. Every output sums its k in a fixed order whatever the tile it falls in.
#include "common.h"
#include "rotary.h"

typedef __bf16 hp_bf8 __attribute__((ext_vector_type(8)));
typedef __bf16 hp_bf4 __attribute__((ext_vector_type(4)));
typedef float hp_f4 __attribute__((ext_vector_type(4)));

template <typename T>
__global__ void latent_norm_cache_kernel(const float* __restrict__ proj, int64_t stride, int q_off, int q_rank, int c_off,
                                         int rank, const float* __restrict__ q_weight, const float* __restrict__ c_weight,
                                         float eps, T* __restrict__ q_out, const int* __restrict__ slots,
                                         T* __restrict__ k_pages, T* __restrict__ v_pages, int page_size, int rot,
                                         const float* __restrict__ inv_freq, const int* __restrict__ positions) {
  __shared__ float scratch[2][16];
  const int64_t row = blockIdx.x;
  const float* pr = proj + row * stride;
  float sq = 0.f, sc = 0.f;
  for (int i = threadIdx.x; i < q_rank; i += blockDim.x) sq += pr[q_off + i] * pr[q_off + i];
  for (int i = threadIdx.x; i < rank; i += blockDim.x) sc += pr[c_off + i] * pr[c_off + i];
  sq = wave_sum(sq);
  sc = wave_sum(sc);
  if (threadIdx.x % DLI_WAVE == 0) {
    scratch[0][threadIdx.x / DLI_WAVE] = sq;
    scratch[1][threadIdx.x / DLI_WAVE] = sc;
  }
  __syncthreads();
  sq = sc = 0.f;
  for (int w = 0; w < (int)blockDim.x / DLI_WAVE; ++w) {     // same order in every thread
    sq += scratch[0][w];
    sc += scratch[1][w];
  }
  const float rq = 1.f / sqrtf(sq / (float)q_rank + eps);
  for (int i = threadIdx.x; i < q_rank; i += blockDim.x)
    q_out[row * q_rank + i] = from_f32<T>(q_weight[i] * (pr[q_off + i] * rq));
  if (rank == 0) return;
  const float rc = 1.f / sqrtf(sc / (float)rank + eps);
  const int slot = slots[row];
  if (slot < 0) return;                                // a padding row: nothing is cached
  const int64_t page = slot / page_size;
  const int off = slot % page_size;
  T* key = k_pages + (page * page_size + off) * (rank + rot);
  for (int i = threadIdx.x; i < rank; i += blockDim.x) {
    const T c = from_f32<T>(c_weight[i] * (pr[c_off + i] * rc));
    key[i] = c;
    if (v_pages != nullptr) v_pages[(page * rank + i) * page_size + off] = c;
  }
  const float* kr = pr + c_off + rank;
  for (int i = threadIdx.x; i < rot / 2; i += blockDim.x) {
    float cs, sn;
    rotary_cos_sin((float)positions[row], inv_freq[i], &cs, &sn);
    const float u = kr[i], v = kr[i + rot / 2];
    key[rank + i] = from_f32<T>(u * cs - v * sn);
    key[rank + rot / 2 + i] = from_f32<T>(v * cs + u * sn);
  }
}

struct HeadProductArgs {
  const void* x; int64_t x_stride; int x_head;       // rows; a head's x begins at h * x_head
  const void* w; int m, k;                           // [heads][m][k]
  void* out; int64_t out_stride; int out_head;       // a head's result begins at h * out_head
  const float* gate; int64_t gate_stride; int gate_per_head;
  int rows, heads;
  int rot; const float* inv_freq; const int* positions;   // rot > 0: x[h][k ..] rotated to out[h][m ..]
};

__device__ __forceinline__ float hp_gate(const HeadProductArgs& p, int64_t row, int head, int n) {
  if (p.gate == nullptr) return 1.f;
  const float g = p.gate[row * p.gate_stride + (p.gate_per_head ? head : head * p.m + n)];
  return 1.f / (1.f + expf(-g));
}

// The rotated tails of `count` rows from r0 on, by all threads of the workgroup.
template <typename T>
__device__ __forceinline__ void hp_rotate(const HeadProductArgs& p, int head, int r0, int count) {
  const int half = p.rot / 2;
  for (int idx = threadIdx.x; idx < count * half; idx += blockDim.x) {
    const int r = r0 + idx / half, i = idx % half;
    if (r >= p.rows) continue;
    const T* src = (const T*)p.x + (int64_t)r * p.x_stride + (int64_t)head * p.x_head + p.k;
    T* dst = (T*)p.out + (int64_t)r * p.out_stride + (int64_t)head * p.out_head + p.m;
    float cs, sn;
    rotary_cos_sin((float)p.positions[r], p.inv_freq[i], &cs, &sn);
    const float u = to_f32(src[i]), v = to_f32(src[i + half]);
    dst[i] = from_f32<T>(u * cs - v * sn);
    dst[i + half] = from_f32<T>(v * cs + u * sn);
  }
}

#define HP_BM 16
#define HP_BN 64
#define HP_BK 32

// A workgroup: 16 rows x 64 outputs of one head; a thread one row and four outputs (tx, tx+16, ...). The last
// z is the rotation's.
template <typename T>
__global__ __launch_bounds__(256) void head_products_kernel(HeadProductArgs p) {
  __shared__ float xs[HP_BM][HP_BK + 1];
  __shared__ float ws[HP_BN][HP_BK + 1];
  const int tid = threadIdx.x, tx = tid % 16, ty = tid / 16;
  const int r0 = blockIdx.x * HP_BM, head = blockIdx.y, n0 = blockIdx.z * HP_BN;
  const int m = p.m, k = p.k, rows = p.rows;
  if (n0 >= m) {
    hp_rotate<T>(p, head, r0, HP_BM);
    return;
  }
  const T* wh = (const T*)p.w + (int64_t)head * m * k;
  const T* x = (const T*)p.x + (int64_t)head * p.x_head;
  float acc[4] = {0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < k; k0 += HP_BK) {
    __syncthreads();
    for (int idx = tid; idx < HP_BM * HP_BK; idx += 256) {
      const int r = idx / HP_BK, c = idx - r * HP_BK;
      xs[r][c] = (r0 + r < rows && k0 + c < k) ? to_f32(x[(int64_t)(r0 + r) * p.x_stride + k0 + c]) : 0.f;
    }
    for (int idx = tid; idx < HP_BN * HP_BK; idx += 256) {
      const int r = idx / HP_BK, c = idx - r * HP_BK;
      ws[r][c] = (n0 + r < m && k0 + c < k) ? to_f32(wh[(int64_t)(n0 + r) * k + k0 + c]) : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int c = 0; c < HP_BK; ++c) {
      const float a = xs[ty][c];
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[j] = fmaf(a, ws[tx + 16 * j][c], acc[j]);
    }
  }
  const int r = r0 + ty;
  if (r >= rows) return;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int n = n0 + tx + 16 * j;
    if (n >= m) continue;
    ((T*)p.out)[(int64_t)r * p.out_stride + (int64_t)head * p.out_head + n] = from_f32<T>(acc[j] * hp_gate(p, r, head, n));
  }
}

// On the matrix cores, in transposed form, out^T = M_h x^T (v_mfma_f32_16x16x32_bf16: lane l supplies row l%16 of
// either operand and the k-indices 8 (l/16) .. + 7). A wave takes 16 MB outputs of 16 RB rows of one head, every operand
// straight from memory, 16 bytes a lane. Which output is which row of a product is free: output
// n0 + 4 MB (j/4) + 4 a + j%4 is row j of product a, so a lane ends with 4 MB neighbouring outputs of one row.
template <int MB, int RB, int WAVES>
__global__ __launch_bounds__(64 * WAVES) void head_products_mfma_kernel(HeadProductArgs p) {
  const int lane = threadIdx.x % 64, wave = threadIdx.x / 64, col = lane & 15, grp = lane >> 4;
  const int head = blockIdx.y, n0 = blockIdx.z * 16 * MB;
  if (n0 >= p.m) {
    hp_rotate<bf16_t>(p, head, blockIdx.x * 16 * RB * WAVES, 16 * RB * WAVES);
    return;
  }
  const int r0 = (blockIdx.x * WAVES + wave) * 16 * RB;
  if (r0 >= p.rows) return;
  const bf16_t* wh = (const bf16_t*)p.w + (int64_t)head * p.m * p.k;
  const bf16_t* wr[MB];
  const bf16_t* xr[RB];
#pragma unroll
  for (int b = 0; b < MB; ++b) wr[b] = wh + (int64_t)min(n0 + 4 * MB * (col / 4) + 4 * b + col % 4, p.m - 1) * p.k;
#pragma unroll
  for (int b = 0; b < RB; ++b)
    xr[b] = (const bf16_t*)p.x + (int64_t)min(r0 + 16 * b + col, p.rows - 1) * p.x_stride + (int64_t)head * p.x_head;
  hp_f4 acc[MB][RB];
#pragma unroll
  for (int a = 0; a < MB; ++a)
#pragma unroll
    for (int b = 0; b < RB; ++b) acc[a][b] = hp_f4{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < p.k; k0 += 32) {
    const int at = k0 + 8 * grp;
    const bool in = at < p.k;                       // (k is a multiple of 8: eight k are inside or outside together)
    hp_bf8 wv[MB], xv[RB];
#pragma unroll
    for (int b = 0; b < MB; ++b) wv[b] = *reinterpret_cast<const hp_bf8*>(wr[b] + (in ? at : 0));
#pragma unroll
    for (int b = 0; b < RB; ++b) {
      xv[b] = *reinterpret_cast<const hp_bf8*>(xr[b] + (in ? at : 0));
      if (!in) xv[b] = hp_bf8{};
    }
    if (!in)
#pragma unroll
      for (int b = 0; b < MB; ++b) wv[b] = hp_bf8{};
#pragma unroll
    for (int a = 0; a < MB; ++a)
#pragma unroll
      for (int b = 0; b < RB; ++b) acc[a][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv[a], xv[b], acc[a][b], 0, 0, 0);
  }
#pragma unroll
  for (int b = 0; b < RB; ++b) {
    const int r = r0 + 16 * b + col;
    if (r >= p.rows) continue;
    bf16_t* o = (bf16_t*)p.out + (int64_t)r * p.out_stride + (int64_t)head * p.out_head;
    const float g1 = p.gate_per_head ? hp_gate(p, r, head, 0) : 1.f;
#pragma unroll
    for (int a = 0; a < MB; ++a) {
      const int n = n0 + 4 * MB * grp + 4 * a;
      if (n >= p.m) continue;                       // (m is a multiple of four)
      hp_bf4 y;
#pragma unroll
      for (int i = 0; i < 4; ++i) y[i] = (bf16_t)(acc[a][b][i] * (p.gate_per_head ? g1 : hp_gate(p, r, head, n + i)));
      *reinterpret_cast<hp_bf4*>(o + n) = y;
    }
  }
}

extern "C" {

int dli_latent_norm_cache(const float* proj, int64_t stride, int q_off, int q_rank, int c_off, int rank,
                          const float* q_weight, const float* c_weight, float eps, void* q_out, const int* slots,
                          void* k_pages, void* v_pages, int rows, int page_size, int rot, const float* inv_freq,
                          const int* positions, int is_bf16, hipStream_t stream) {
  if (rows <= 0) return DLI_OK;
  if (q_rank <= 0 || rank < 0 || page_size <= 0 || q_off < 0 || c_off < 0 || q_off + q_rank > stride || rot < 0 || rot % 2 ||
      c_off + rank + rot > stride || (rank > 0 && (k_pages == nullptr || slots == nullptr)) ||
      (rot > 0 && (rank == 0 || inv_freq == nullptr || positions == nullptr || v_pages != nullptr)))
    return DLI_ERR_ARGUMENT;
  const int widest = q_rank > rank ? q_rank : rank;
  const int threads = widest >= 1024 ? 512 : widest >= 256 ? 256 : 64;
  if (is_bf16)
    latent_norm_cache_kernel<bf16_t><<<rows, threads, 0, stream>>>(
        proj, stride, q_off, q_rank, c_off, rank, q_weight, c_weight, eps, (bf16_t*)q_out, slots, (bf16_t*)k_pages,
        (bf16_t*)v_pages, page_size, rot, inv_freq, positions);
  else
    latent_norm_cache_kernel<float><<<rows, threads, 0, stream>>>(
        proj, stride, q_off, q_rank, c_off, rank, q_weight, c_weight, eps, (float*)q_out, slots, (float*)k_pages,
        (float*)v_pages, page_size, rot, inv_freq, positions);
  return dli_launch_status();
}

int dli_head_products(const void* x, int64_t x_stride, int x_head, const void* w, void* out, int64_t out_stride, int out_head,
                      const float* gate, int64_t gate_stride, int gate_per_head, int rows, int heads, int m, int k, int rot,
                      const float* inv_freq, const int* positions, int is_bf16, hipStream_t stream) {
  if (rows <= 0) return DLI_OK;
  if (heads <= 0 || heads > 65535 || m <= 0 || k <= 0 || rot < 0 || rot % 2 || x_head < k + rot || out_head < m + rot ||
      x_stride < (int64_t)heads * x_head || out_stride < (int64_t)heads * out_head ||
      (rot > 0 && (inv_freq == nullptr || positions == nullptr)) ||
      (gate != nullptr && gate_stride < (gate_per_head ? (int64_t)heads : (int64_t)heads * m)))
    return DLI_ERR_ARGUMENT;
  HeadProductArgs p;
  p.x = x; p.x_stride = x_stride; p.x_head = x_head; p.w = w; p.m = m; p.k = k; p.out = out; p.out_stride = out_stride;
  p.out_head = out_head; p.gate = gate; p.gate_stride = gate_stride; p.gate_per_head = gate_per_head; p.rows = rows;
  p.heads = heads; p.rot = rot; p.inv_freq = inv_freq; p.positions = positions;
  const bool mfma = is_bf16 && k % 8 == 0 && m % 4 == 0 && x_head % 8 == 0 && x_stride % 8 == 0 && out_head % 4 == 0 &&
                    out_stride % 4 == 0 && ((uintptr_t)x | (uintptr_t)w) % 16 == 0 && (uintptr_t)out % 8 == 0;
#define HP_GRID(RROWS, OUTS) dim3((rows + (RROWS)-1) / (RROWS), heads, (m + (OUTS)-1) / (OUTS) + (rot > 0))
  if (mfma && (m + 15) / 16 < 65534) {
    if (rows <= 16) head_products_mfma_kernel<1, 1, 1><<<HP_GRID(16, 16), 64, 0, stream>>>(p);
    else if (rows <= 64) head_products_mfma_kernel<2, 1, 4><<<HP_GRID(64, 32), 256, 0, stream>>>(p);
    else head_products_mfma_kernel<4, 4, 4><<<HP_GRID(256, 64), 256, 0, stream>>>(p);
    return dli_launch_status();
  }
  const dim3 grid = HP_GRID(HP_BM, HP_BN);
  if (grid.z > 65535) return DLI_ERR_ARGUMENT;
  if (is_bf16) head_products_kernel<bf16_t><<<grid, 256, 0, stream>>>(p);
  else head_products_kernel<float><<<grid, 256, 0, stream>>>(p);
#undef HP_GRID
  return dli_launch_status();
}

}  // extern "C"
