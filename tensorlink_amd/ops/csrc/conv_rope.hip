// Short causal convolution over time + rotate-half positions + page
// scatter in one kernel (gfx950).
//
// Columns [col, col + n_heads*D) of the fused projection (bf16 or fp32)
// pass a per-channel convolution with K taps,
//     y_t[c] = sum_j taps[c][j] u_(t-K+1+j)[c]  (+ bias[c], silu),
// whose inputs before the step's first token come from the sequence's
// history [slots, K-1, N] (fp32; zeros when the sequence has no cached
// tokens). The first rot_dims dimensions of every head are then rotated by
// the token's position: pair (i, i + rot_dims/2), angle pos * freqs[i]
// formed in double, cos and sin times `mult`. The first n_heads -
// pool_heads heads are written densely in fp32 (queries, or the inputs of a
// recurrence); the last pool_heads heads go to the tokens' page rows of
// `pool` (rotated) and, when given, of `raw_pool` (the unrotated
// convolution output: a value pool that shares the key projection).
//
// One block per tile of <= TILE tokens of one sequence (with few tiles the
// work items of a tile are spread over several blocks). A work item is a
// rotated pair or a single unrotated channel, so rotation needs no
// exchange between threads; the tile's cos/sin table is built once in LDS
// and shared by all heads. TILE >= K-1, so only the block of a portion's
// first tile reads the old history; the same block writes the new one
// after a barrier.

#include "common.hpp"

namespace {

constexpr int BLOCK = 256;
constexpr int TILE = 8;
constexpr int PAGE = 128;
constexpr int MAXK = 9;

template <typename T> DEVINLINE float ldf(const T* p, int64_t i);
template <> DEVINLINE float ldf<float>(const float* p, int64_t i) { return p[i]; }
template <> DEVINLINE float ldf<bf16>(const bf16* p, int64_t i) { return bf2f(p[i]); }
template <typename T> DEVINLINE void stf(T* p, int64_t i, float v);
template <> DEVINLINE void stf<float>(float* p, int64_t i, float v) { p[i] = v; }
template <> DEVINLINE void stf<bf16>(bf16* p, int64_t i, float v) { p[i] = f2bf(v); }

DEVINLINE float silu_f(float z) { return z / (1.f + expf(-z)); }

template <typename T>
__global__ __launch_bounds__(BLOCK) void conv_rope_rows_kernel(
    const T* __restrict__ src, int ld, int col, int n_heads, int D,
    const float* __restrict__ taps, const float* __restrict__ bias,
    int act_silu, float* __restrict__ hist, int K, int rot_dims,
    const double* __restrict__ freqs, float mult,
    const int* __restrict__ tiles, const int* __restrict__ cu,
    const int* __restrict__ slots, const int* __restrict__ pos0,
    const int* __restrict__ table, int P, float* __restrict__ out,
    T* __restrict__ pool, T* __restrict__ raw_pool, int pool_heads) {
  extern __shared__ float cs[];     // [TILE][half][2]
  const int seq = tiles[blockIdx.x * 4 + 0];
  const int tok0 = tiles[blockIdx.x * 4 + 1];
  const int n = tiles[blockIdx.x * 4 + 2];
  const int p0 = tiles[blockIdx.x * 4 + 3];
  const int c0 = cu[seq], ntot = cu[seq + 1] - c0;
  const bool first = tok0 == c0;
  const bool fresh = pos0[seq] == 0;
  const int half = rot_dims / 2;
  const int N = n_heads * D;
  const int dense = n_heads - pool_heads;
  for (int i = threadIdx.x; i < n * half; i += BLOCK) {
    const int t = i / half, p = i - t * half;
    const double ang = (double)(p0 + t) * freqs[p];
    cs[i * 2 + 0] = (float)(cos(ang) * (double)mult);
    cs[i * 2 + 1] = (float)(sin(ang) * (double)mult);
  }
  __syncthreads();
  float* hs = hist + (int64_t)slots[seq] * (K - 1) * N;
  const int iph = D - half;         // work items per head
  const int* tab = table + (int64_t)seq * P;
  // few tiles (decoding): the work items are spread over gridDim.y blocks
  const int e_first = blockIdx.y * BLOCK + threadIdx.x;
  const int e_step = gridDim.y * BLOCK;
  for (int e = e_first; e < n_heads * iph; e += e_step) {
    const int hd = e / iph, r = e - hd * iph;
    const bool pair = r < half;
    const int d0 = pair ? r : r + half;
    const int ch0 = hd * D + d0, ch1 = ch0 + half;
    // taps and the sliding window are aligned at the END of fixed-size
    // arrays (leading entries zero), so every index is static
    float w0[MAXK], w1[MAXK], u0[MAXK - 1], u1[MAXK - 1];
#pragma unroll
    for (int m = 0; m < MAXK; ++m) {
      const int j = m - (MAXK - K);
      w0[m] = j >= 0 ? taps[(int64_t)ch0 * K + j] : 0.f;
      w1[m] = (pair && j >= 0) ? taps[(int64_t)ch1 * K + j] : 0.f;
    }
#pragma unroll
    for (int m = 0; m < MAXK - 1; ++m) {
      const int j = m - (MAXK - K);
      float a = 0.f, b = 0.f;
      if (j >= 0) {
        const int row = tok0 - (K - 1) + j;
        if (row >= c0) {
          a = ldf<T>(src, (int64_t)row * ld + col + ch0);
          if (pair) b = ldf<T>(src, (int64_t)row * ld + col + ch1);
        } else if (!fresh) {
          const int64_t hr = (int64_t)(K - 1 + row - c0) * N;
          a = hs[hr + ch0];
          if (pair) b = hs[hr + ch1];
        }
      }
      u0[m] = a;
      u1[m] = b;
    }
    const float b0 = bias ? bias[ch0] : 0.f;
    const float b1 = (bias && pair) ? bias[ch1] : 0.f;
    for (int i = 0; i < n; ++i) {
      const int64_t ro = (int64_t)(tok0 + i) * ld + col;
      const float c0v = ldf<T>(src, ro + ch0);
      const float c1v = pair ? ldf<T>(src, ro + ch1) : 0.f;
      float a0 = b0 + w0[MAXK - 1] * c0v, a1 = b1 + w1[MAXK - 1] * c1v;
#pragma unroll
      for (int m = 0; m < MAXK - 1; ++m) {
        a0 += w0[m] * u0[m];
        a1 += w1[m] * u1[m];
      }
#pragma unroll
      for (int m = 0; m < MAXK - 2; ++m) {
        u0[m] = u0[m + 1];
        u1[m] = u1[m + 1];
      }
      u0[MAXK - 2] = c0v;
      u1[MAXK - 2] = c1v;
      if (act_silu) {
        a0 = silu_f(a0);
        a1 = silu_f(a1);
      }
      float x0 = a0, x1 = a1;
      if (pair) {
        const float c = cs[(i * half + r) * 2], s = cs[(i * half + r) * 2 + 1];
        x0 = a0 * c - a1 * s;
        x1 = a1 * c + a0 * s;
      }
      const int tok = tok0 + i;
      if (hd < dense) {
        float* o = out + (int64_t)tok * dense * D + hd * D;
        o[d0] = x0;
        if (pair) o[d0 + half] = x1;
      } else {
        const int pos = p0 + i;
        const int64_t prow =
            (((int64_t)tab[pos / PAGE] * pool_heads + (hd - dense)) * PAGE +
             (pos % PAGE)) * D;
        stf<T>(pool, prow + d0, x0);
        if (pair) stf<T>(pool, prow + d0 + half, x1);
        if (raw_pool) {
          stf<T>(raw_pool, prow + d0, a0);
          if (pair) stf<T>(raw_pool, prow + d0 + half, a1);
        }
      }
    }
  }
  if (!first || K <= 1) return;
  __syncthreads();       // every read of the old history is done
  // a block updates the channels of its own work items
  for (int e = e_first; e < n_heads * iph; e += e_step) {
    const int hd = e / iph, r = e - hd * iph;
    const bool pair = r < half;
    const int ch0 = hd * D + (pair ? r : r + half);
    for (int k = 0; k < (pair ? 2 : 1); ++k) {
      const int c = ch0 + k * half;
      for (int r2 = 0; r2 < K - 1; ++r2) {
        const int rr = ntot - (K - 1) + r2;
        float v;
        if (rr >= 0)
          v = ldf<T>(src, (int64_t)(c0 + rr) * ld + col + c);
        else    // ascending: source index r2 + ntot is not yet overwritten
          v = fresh ? 0.f : hs[(int64_t)(r2 + ntot) * N + c];
        hs[(int64_t)r2 * N + c] = v;
      }
    }
  }
}

struct alignas(8) bf16x4 {
  bf16 v[4];
};
DEVINLINE void ld4(const float* p, float (&o)[4]) {
  const float4 x = *reinterpret_cast<const float4*>(p);
  o[0] = x.x;
  o[1] = x.y;
  o[2] = x.z;
  o[3] = x.w;
}
DEVINLINE void ld4(const bf16* p, float (&o)[4]) {
  const bf16x4 x = *reinterpret_cast<const bf16x4*>(p);
#pragma unroll
  for (int e = 0; e < 4; ++e) o[e] = bf2f(x.v[e]);
}

// The same without rotation and without pools, N, ld and col multiples of 4:
// a thread owns four channels of a tile, whose rows are all in flight before
// the first product.
template <typename T, int K>
__global__ __launch_bounds__(BLOCK) void conv_dense_kernel(
    const T* __restrict__ src, int ld, int col, int N,
    const float* __restrict__ taps, const float* __restrict__ bias,
    int act_silu, float* __restrict__ hist, const int* __restrict__ tiles,
    const int* __restrict__ cu, const int* __restrict__ slots,
    const int* __restrict__ pos0, float* __restrict__ out) {
  const int c = (blockIdx.y * BLOCK + threadIdx.x) * 4;
  if (c >= N) return;                // no barrier in this kernel
  const int seq = tiles[blockIdx.x * 4 + 0];
  const int tok0 = tiles[blockIdx.x * 4 + 1];
  const int n = tiles[blockIdx.x * 4 + 2];
  const int c0 = cu[seq], ntot = cu[seq + 1] - c0;
  const bool first = tok0 == c0, fresh = pos0[seq] == 0;
  float* hs = hist + (int64_t)slots[seq] * (K - 1) * N + c;
  const T* sc = src + col + c;
  float u[K - 1 + TILE][4];          // rows tok0 - (K-1) .. tok0 + TILE - 1
#pragma unroll
  for (int i = 0; i < TILE; ++i)
    ld4(sc + (int64_t)(tok0 + min(i, n - 1)) * ld, u[K - 1 + i]);
  if (!first) {                      // TILE >= K - 1: all in the portion
#pragma unroll
    for (int j = 0; j < K - 1; ++j)
      ld4(sc + (int64_t)(tok0 - (K - 1) + j) * ld, u[j]);
  } else {
#pragma unroll
    for (int j = 0; j < K - 1; ++j) {
      if (fresh) {
#pragma unroll
        for (int e = 0; e < 4; ++e) u[j][e] = 0.f;
      } else {
        ld4(hs + (int64_t)j * N, u[j]);
      }
    }
  }
  float w[4 * K], b[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int j = 0; j < K; ++j) {
    float x[4];
    ld4(taps + (int64_t)c * K + 4 * j, x);
#pragma unroll
    for (int e = 0; e < 4; ++e) w[4 * j + e] = x[e];
  }
  if (bias) ld4(bias + c, b);
#pragma unroll
  for (int i = 0; i < TILE; ++i) {
    if (i < n) {
      float a[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        a[e] = b[e];
#pragma unroll
        for (int j = 0; j < K; ++j) a[e] += w[e * K + j] * u[i + j][e];
        if (act_silu) a[e] = silu_f(a[e]);
      }
      *reinterpret_cast<float4*>(out + (int64_t)(tok0 + i) * N + c) =
          make_float4(a[0], a[1], a[2], a[3]);
    }
  }
  if (!first) return;
  // the portion's last K-1 rows; a thread reads and writes its own channels
#pragma unroll
  for (int r = 0; r < K - 1; ++r) {
    const int rr = ntot - (K - 1) + r;
    float v[4] = {0.f, 0.f, 0.f, 0.f};
    if (rr >= 0)
      ld4(sc + (int64_t)(c0 + rr) * ld, v);
    else if (!fresh)   // ascending: source row r + ntot is not overwritten yet
      ld4(hs + (int64_t)(r + ntot) * N, v);
    *reinterpret_cast<float4*>(hs + (int64_t)r * N) =
        make_float4(v[0], v[1], v[2], v[3]);
  }
}

template <typename T>
void launch_dense(const T* src, int ld, int col, int N, const float* taps,
                  const float* bias, int act_silu, float* hist, int K,
                  const int* tiles, int n_tiles, const int* cu,
                  const int* slots, const int* pos0, float* out,
                  hipStream_t stream) {
  const dim3 grid(n_tiles, (N / 4 + BLOCK - 1) / BLOCK);
#define TL_CD(KK)                                                            \
  case KK:                                                                   \
    hipLaunchKernelGGL((conv_dense_kernel<T, KK>), grid, dim3(BLOCK), 0,     \
                       stream, src, ld, col, N, taps, bias, act_silu, hist,  \
                       tiles, cu, slots, pos0, out);                         \
    break
  switch (K) {
    TL_CD(1);
    TL_CD(2);
    TL_CD(3);
    TL_CD(4);
    TL_CD(5);
    TL_CD(6);
    TL_CD(7);
    TL_CD(8);
    default:
      TL_CD(9);
  }
#undef TL_CD
}

}  // namespace

extern "C" {

int tl_conv_rope_tile() { return TILE; }

// returns 0 on success, 1 if the shape is outside what the kernel serves
int tl_conv_rope_rows(const void* src, int ld, int col, int n_heads, int D,
                      const void* taps, const void* bias, int act_silu,
                      void* hist, int K, int rot_dims, const void* freqs,
                      float mult, const void* tiles, int n_tiles,
                      const void* cu, const void* slots, const void* pos0,
                      const void* table, int P, void* out, void* pool,
                      void* raw_pool, int pool_heads, int is_f32,
                      hipStream_t stream) {
  if (n_tiles <= 0) return 0;
  if (K < 1 || K > MAXK || K - 1 > TILE || (rot_dims & 1) || rot_dims > D)
    return 1;
  const size_t smem = sizeof(float) * 2 * TILE * (size_t)(rot_dims / 2);
  if (smem > 64 * 1024) return 1;
  const int N = n_heads * D;
  if (rot_dims == 0 && pool_heads == 0 && N % 4 == 0 && ld % 4 == 0 &&
      col % 4 == 0) {
    if (is_f32)
      launch_dense<float>((const float*)src, ld, col, N, (const float*)taps,
                          (const float*)bias, act_silu, (float*)hist, K,
                          (const int*)tiles, n_tiles, (const int*)cu,
                          (const int*)slots, (const int*)pos0, (float*)out,
                          stream);
    else
      launch_dense<bf16>((const bf16*)src, ld, col, N, (const float*)taps,
                         (const float*)bias, act_silu, (float*)hist, K,
                         (const int*)tiles, n_tiles, (const int*)cu,
                         (const int*)slots, (const int*)pos0, (float*)out,
                         stream);
    return 0;
  }
  const int items = n_heads * (D - rot_dims / 2);
  const int gy = n_tiles >= 512 ? 1 : min(16, max(1, (items + BLOCK - 1) / BLOCK));
  const dim3 grid(n_tiles, gy);
  if (is_f32)
    hipLaunchKernelGGL(conv_rope_rows_kernel<float>, grid,
                       dim3(BLOCK), smem, stream, (const float*)src, ld, col,
                       n_heads, D, (const float*)taps, (const float*)bias,
                       act_silu, (float*)hist, K, rot_dims,
                       (const double*)freqs, mult, (const int*)tiles,
                       (const int*)cu, (const int*)slots, (const int*)pos0,
                       (const int*)table, P, (float*)out, (float*)pool,
                       (float*)raw_pool, pool_heads);
  else
    hipLaunchKernelGGL(conv_rope_rows_kernel<bf16>, grid,
                       dim3(BLOCK), smem, stream, (const bf16*)src, ld, col,
                       n_heads, D, (const float*)taps, (const float*)bias,
                       act_silu, (float*)hist, K, rot_dims,
                       (const double*)freqs, mult, (const int*)tiles,
                       (const int*)cu, (const int*)slots, (const int*)pos0,
                       (const int*)table, P, (float*)out, (bf16*)pool,
                       (bf16*)raw_pool, pool_heads);
  return 0;
}

}  // extern "C"
