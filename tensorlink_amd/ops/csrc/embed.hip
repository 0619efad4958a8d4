// Token embedding plus a hashed bigram embedding over ragged sequences, and
// thin fp32 projections (gfx950).
//
// tl_bigram_embed: X[t] = embed[tok_t] + table[row_t] in fp32, row_t =
// (tok_(t-1) * mul_prev + tok_t * mul_cur) mod n, the table's row n for a
// sequence's first token. The token before a portion comes from the
// sequence's slot (int32), which is left holding the portion's last token.
// One block per token; the block of a portion's first token is the only one
// that touches the slot, and one thread of it reads before it writes.
//
// tl_thin_linear: out = h W^T + b in fp32 for few rows and few outputs
// (gates, step sizes, router logits): h and W bf16 or fp32, one wave per
// four outputs of a token.

#include "common.hpp"

namespace {

constexpr int BLOCK = 256;
constexpr int NWAVE = BLOCK / WAVE_SIZE;

template <typename T> DEVINLINE float ldf(const T* p);
template <> DEVINLINE float ldf<float>(const float* p) { return *p; }
template <> DEVINLINE float ldf<bf16>(const bf16* p) { return bf2f(*p); }

struct alignas(8) bf16x4 {
  bf16 v[4];
};
DEVINLINE float4 ld4(const float* p) {
  return *reinterpret_cast<const float4*>(p);
}
DEVINLINE float4 ld4(const bf16* p) {
  const bf16x4 x = *reinterpret_cast<const bf16x4*>(p);
  return make_float4(bf2f(x.v[0]), bf2f(x.v[1]), bf2f(x.v[2]), bf2f(x.v[3]));
}

// an id outside the vocabulary reads the nearest row
template <typename T>
__global__ __launch_bounds__(BLOCK) void bigram_embed_kernel(
    const int64_t* __restrict__ tokens, const T* __restrict__ embed,
    const T* __restrict__ table, int* __restrict__ prev,
    const int* __restrict__ tok_seq, const int* __restrict__ cu,
    const int* __restrict__ slots, const int* __restrict__ pos0,
    float* __restrict__ X, int W, int64_t vocab, int64_t n, int64_t mul_prev,
    int64_t mul_cur) {
  __shared__ int64_t row_s;
  const int64_t t = blockIdx.x;
  int64_t cur = tokens[t];
  cur = cur < 0 ? 0 : (cur >= vocab ? vocab - 1 : cur);
  if (threadIdx.x == 0) {
    const int b = tok_seq[t];
    int64_t row = n;
    if (t > cu[b]) {
      row = (tokens[t - 1] * mul_prev + cur * mul_cur) % n;
    } else {
      if (pos0[b] > 0)
        row = ((int64_t)prev[slots[b]] * mul_prev + cur * mul_cur) % n;
      prev[slots[b]] = (int)tokens[cu[b + 1] - 1];
    }
    row_s = row < 0 ? row + n : row;
  }
  __syncthreads();
  const T* e = embed + cur * W;
  const T* g = table + row_s * W;
  float* x = X + t * W;
  if (W % 4 == 0) {
    for (int c = threadIdx.x * 4; c < W; c += BLOCK * 4) {
      const float4 a = ld4(e + c), b = ld4(g + c);
      *reinterpret_cast<float4*>(x + c) =
          make_float4(a.x + b.x, a.y + b.y, a.z + b.z, a.w + b.w);
    }
  } else {
    for (int c = threadIdx.x; c < W; c += BLOCK)
      x[c] = ldf<T>(e + c) + ldf<T>(g + c);
  }
}

// grid (T, ceil(N / 16)): a wave computes four outputs
template <typename T, bool VEC>
__global__ __launch_bounds__(BLOCK) void thin_linear_kernel(
    const T* __restrict__ h, const T* __restrict__ w,
    const float* __restrict__ bias, float* __restrict__ out, int W, int N) {
  const int64_t t = blockIdx.x;
  const int lane = threadIdx.x & (WAVE_SIZE - 1);
  const int n0 = (blockIdx.y * NWAVE + threadIdx.x / WAVE_SIZE) * 4;
  if (n0 >= N) return;
  const T* hr = h + t * W;
  const T* wr[4];
  float s[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int u = 0; u < 4; ++u) wr[u] = w + (int64_t)min(n0 + u, N - 1) * W;
  if (VEC) {
#pragma unroll 2
    for (int c = lane * 4; c < W; c += WAVE_SIZE * 4) {
      const float4 x = ld4(hr + c);
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const float4 y = ld4(wr[u] + c);
        s[u] += x.x * y.x + x.y * y.y + x.z * y.z + x.w * y.w;
      }
    }
  } else {
    for (int c = lane; c < W; c += WAVE_SIZE) {
      const float x = ldf<T>(hr + c);
#pragma unroll
      for (int u = 0; u < 4; ++u) s[u] += x * ldf<T>(wr[u] + c);
    }
  }
#pragma unroll
  for (int u = 0; u < 4; ++u) {
    const float v = wave_reduce_sum(s[u]);
    if (lane == 0 && n0 + u < N)
      out[t * N + n0 + u] = v + (bias ? bias[n0 + u] : 0.f);
  }
}

}  // namespace

extern "C" {

void tl_bigram_embed(const void* tokens, const void* embed, const void* table,
                     void* prev, const void* tok_seq, const void* cu,
                     const void* slots, const void* pos0, void* X, int64_t T,
                     int W, int64_t vocab, int64_t n, int64_t mul_prev,
                     int64_t mul_cur, int is_f32, hipStream_t stream) {
  if (T <= 0) return;
  dim3 grid((unsigned)T), block(BLOCK);
#define TL_BE(TT)                                                           \
  hipLaunchKernelGGL(bigram_embed_kernel<TT>, grid, block, 0, stream,       \
                     (const int64_t*)tokens, (const TT*)embed,              \
                     (const TT*)table, (int*)prev, (const int*)tok_seq,     \
                     (const int*)cu, (const int*)slots, (const int*)pos0,   \
                     (float*)X, W, vocab, n, mul_prev, mul_cur)
  if (is_f32) TL_BE(float);
  else TL_BE(bf16);
#undef TL_BE
}

void tl_thin_linear(const void* h, const void* w, const void* bias, void* out,
                    int64_t T, int W, int N, int is_f32, hipStream_t stream) {
  if (T <= 0 || N <= 0) return;
  dim3 grid((unsigned)T, (N + 4 * NWAVE - 1) / (4 * NWAVE)), block(BLOCK);
#define TL_TL(TT, VV)                                                        \
  hipLaunchKernelGGL((thin_linear_kernel<TT, VV>), grid, block, 0, stream,   \
                     (const TT*)h, (const TT*)w, (const float*)bias,         \
                     (float*)out, W, N)
  if (is_f32) {
    if (W % 4 == 0) TL_TL(float, true);
    else TL_TL(float, false);
  } else {
    if (W % 4 == 0) TL_TL(bf16, true);
    else TL_TL(bf16, false);
  }
#undef TL_TL
}

}  // extern "C"
