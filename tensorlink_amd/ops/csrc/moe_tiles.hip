// Grouped expert products with stacked experts on MFMA (gfx950, bf16): the
// two ends of the range around moe_gemm.hip.
//
// out[p][n] = sum_k x[tok ? tok[p] : p][k] w[e][n][k] for the pairs p of
// expert e (seg[e] <= p < seg[e + 1]).
//
// tl_moe_tiles (prompts): 128 pairs x 128 columns per block, four waves of
// 64 x 64. Both panels go to LDS by direct loads (global_load_lds, rows
// gathered through tok), double-buffered over 64-wide k steps; the 16-byte
// slots of a row are permuted by the row number on the source address, and
// the fragment reads apply the same permutation. The tile list is implicit:
// the grid has an upper bound of tiles (P / 128 + E), a block finds its
// expert with a wave-wide scan over the segments and leaves if there is
// none. Consecutive tiles go to one XCD, columns first, so an expert's
// weights and a tile's rows are read from that XCD's L2. The weight is the
// A operand, so a lane ends with four neighbouring columns of one row. The
// k order per row is that of moe_gemm.hip.
//
// tl_moe_rows (decoding): few pairs per expert. A block covers 16 columns of
// one expert; its four waves take a quarter of K each, straight from global
// memory (all loads of a quarter are in flight before the first product),
// and meet in LDS.

#include "common.hpp"

namespace {

constexpr int BLOCK = 256;
constexpr int BM = 128, BN = 128, BK = 64;

using f32x4 = __attribute__((ext_vector_type(4))) float;
typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));

struct alignas(8) bf16x4 {
  bf16 v[4];
};

__global__ __launch_bounds__(BLOCK, 2) void moe_tile_kernel(
    const bf16* __restrict__ x, const int* __restrict__ tok,
    const int* __restrict__ seg, const bf16* __restrict__ w,
    bf16* __restrict__ out, int E, int N, int K, int n_tiles) {
  __shared__ bf16 lds[2][BM + BN][BK];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  // blocks go round-robin over the 8 XCDs: give each a contiguous stretch
  const int per = gridDim.x / 8;                  // grid is a multiple of 8
  const int id = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
  const int nt = (N + BN - 1) / BN;
  const int mt = id / nt, n0 = (id - mt * nt) * BN;
  if (mt >= n_tiles) return;
  // expert and row tile of the mt-th tile
  int e = -1, mb = 0, run = 0;
  for (int eb = 0; eb < E; eb += 64) {
    const int ee = eb + lane;
    const int c =
        ee < E ? (seg[ee + 1] - seg[ee] + BM - 1) / BM : 0;
    int inc = c;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const int o = __shfl_up(inc, off, WAVE_SIZE);
      if (lane >= off) inc += o;
    }
    const int tot = __shfl(inc, 63, WAVE_SIZE);
    if (mt < run + tot) {
      const unsigned long long m = __ballot(mt < run + inc);
      const int l = __ffsll((long long)m) - 1;
      e = eb + l;
      mb = mt - run - __shfl(inc - c, l, WAVE_SIZE);
      break;
    }
    run += tot;
  }
  if (e < 0) return;
  const int m0 = seg[e] + mb * BM;
  const int rows = min(BM, seg[e + 1] - m0);
  const bf16* we = w + (int64_t)e * N * K;

  // wave w loads the 8-row groups 8w .. 8w+7 of the 32 (x rows, then w rows)
  const int l8 = lane >> 3, c8 = lane & 7;
  const bf16* src[8];
#pragma unroll
  for (int g = 0; g < 8; ++g) {
    const int r = (wave * 8 + g) * 8 + l8;
    if (r < BM) {
      const int p = m0 + min(r, rows - 1);
      src[g] = x + (int64_t)(tok ? tok[p] : p) * K;
    } else {
      src[g] = we + (int64_t)min(n0 + r - BM, N - 1) * K;
    }
  }
#define MT_LOAD(bufi, k0)                                                   \
  _Pragma("unroll") for (int g = 0; g < 8; ++g) {                           \
    const int r8 = (wave * 8 + g) * 8;                                      \
    const int kc = min((k0) + (c8 ^ l8) * 8, K - 8);                        \
    __builtin_amdgcn_global_load_lds(                                       \
        (const __attribute__((address_space(1))) void*)(src[g] + kc),       \
        (__attribute__((address_space(3))) void*)(&lds[bufi][r8][0]), 16, 0, \
        0);                                                                 \
  }

  const int col = lane & 15, quad = lane >> 4;
  const int wm = (wave & 1) * 64, wn = (wave >> 1) * 64;
  f32x4 acc[4][4];                       // [n tile][m tile]
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = (f32x4){0.f, 0.f, 0.f, 0.f};

  MT_LOAD(0, 0)
  int buf = 0;
  for (int k0 = 0; k0 < K; k0 += BK) {
    __syncthreads();
    if (k0 + BK < K) { MT_LOAD(buf ^ 1, k0 + BK) }
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      if (k0 + kk * 32 >= K) break;
      bf16x8_t xf[4], wf[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int s = ((kk * 4 + quad) ^ (col & 7)) * 8;
        xf[i] = *reinterpret_cast<const bf16x8_t*>(
            &lds[buf][wm + i * 16 + col][s]);
        wf[i] = *reinterpret_cast<const bf16x8_t*>(
            &lds[buf][BM + wn + i * 16 + col][s]);
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j)
          acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              wf[i], xf[j], acc[i][j], 0, 0, 0);
    }
    buf ^= 1;
  }
#undef MT_LOAD
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int m = wm + j * 16 + col;
    if (m >= rows) continue;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int n = n0 + wn + i * 16 + quad * 4;
      if (n >= N) continue;              // N is a multiple of 64
      bf16x4 o;
#pragma unroll
      for (int r = 0; r < 4; ++r) o.v[r] = f2bf(acc[i][j][r]);
      *reinterpret_cast<bf16x4*>(out + (int64_t)(m0 + m) * N + n) = o;
    }
  }
}

// KS: 32-wide k steps per wave and pass
template <int KS>
__global__ __launch_bounds__(BLOCK) void moe_rows_kernel(
    const bf16* __restrict__ x, const int* __restrict__ tok,
    const int* __restrict__ seg, const bf16* __restrict__ w,
    bf16* __restrict__ out, int N, int K) {
  __shared__ float red[4][16][17];
  const int e = blockIdx.y, n0 = blockIdx.x * 16;
  const int p0 = seg[e], mt = seg[e + 1] - p0;
  if (mt <= 0) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int col = lane & 15, quad = lane >> 4;
  const int steps = K / 32;
  const bf16* wr = w + ((int64_t)e * N + n0 + col) * K + quad * 8;
  for (int mb = 0; mb < mt; mb += 16) {
    const int p = p0 + min(mb + col, mt - 1);
    const bf16* xr = x + (int64_t)(tok ? tok[p] : p) * K + quad * 8;
    f32x4 acc = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int s0 = wave * KS; s0 < steps; s0 += 4 * KS) {
      bf16x8_t wf[KS], xf[KS];
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        const int k = min(s0 + s, steps - 1) * 32;
        wf[s] = *reinterpret_cast<const bf16x8_t*>(wr + k);
        xf[s] = *reinterpret_cast<const bf16x8_t*>(xr + k);
      }
#pragma unroll
      for (int s = 0; s < KS; ++s)
        if (s0 + s < steps)
          acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[s], xf[s], acc, 0,
                                                        0, 0);
    }
    __syncthreads();
#pragma unroll
    for (int r = 0; r < 4; ++r) red[wave][quad * 4 + r][col] = acc[r];
    __syncthreads();
    // thread (row m, column n) of the 16 x 16 tile
    const int m = threadIdx.x >> 4, n = threadIdx.x & 15;
    if (mb + m < mt) {
      float s = 0.f;
#pragma unroll
      for (int u = 0; u < 4; ++u) s += red[u][n][m];
      out[(int64_t)(p0 + mb + m) * N + n0 + n] = f2bf(s);
    }
  }
}

}  // namespace

extern "C" {

// N a multiple of 64, K of 32
void tl_moe_tiles(const void* x, const void* tok, const void* seg,
                  const void* w, void* out, int P, int E, int N, int K,
                  hipStream_t stream) {
  if (P <= 0) return;
  const int tiles = P / BM + E;          // every segment adds at most one
  const int blocks = tiles * ((N + BN - 1) / BN);
  hipLaunchKernelGGL(moe_tile_kernel, dim3((blocks + 7) / 8 * 8), dim3(BLOCK),
                     0, stream, (const bf16*)x, (const int*)tok,
                     (const int*)seg, (const bf16*)w, (bf16*)out, E, N, K,
                     tiles);
}

// N a multiple of 16, K of 32
void tl_moe_rows(const void* x, const void* tok, const void* seg,
                 const void* w, void* out, int P, int E, int N, int K,
                 hipStream_t stream) {
  if (P <= 0) return;
  dim3 grid(N / 16, E), block(BLOCK);
  const int per = (K / 32 + 3) / 4;      // k steps of a wave
#define TL_MR(KS)                                                            \
  hipLaunchKernelGGL(moe_rows_kernel<KS>, grid, block, 0, stream,            \
                     (const bf16*)x, (const int*)tok, (const int*)seg,       \
                     (const bf16*)w, (bf16*)out, N, K)
  if (per <= 1) TL_MR(1);
  else if (per <= 2) TL_MR(2);
  else if (per <= 3) TL_MR(3);
  else if (per <= 4) TL_MR(4);
  else TL_MR(8);
#undef TL_MR
}

}  // extern "C"
