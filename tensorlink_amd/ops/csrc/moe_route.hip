// Routing of a mixture of experts (gfx950): fp32 router logits, selection of
// the largest ones with a softmax over the chosen (or scores from a softmax
// over all experts, chosen with a correction), expert-sorted (token, choice)
// pairs, a grouped product for shapes and dtypes that the MFMA
// kernel (moe_gemm.hip) does not take, and the weighted combine.
//
// The position of a pair inside its expert's segment is handed out by LDS
// atomics, so the order inside a segment may differ between runs; a row of
// the grouped products does not depend on its place, and the combine reads
// the choices of a token in their own order, so results do not.

#include "common.hpp"

namespace {

constexpr int BLOCK = 256;
constexpr int NWAVE = BLOCK / WAVE_SIZE;
constexpr int MAX_TOP = 64;
constexpr int MAX_E = 2048;          // one mask bit per 64 experts and lane
constexpr int TILE = 2048;           // pairs per block of the sort

template <typename T> DEVINLINE float ldf(const T* p);
template <> DEVINLINE float ldf<float>(const float* p) { return *p; }
template <> DEVINLINE float ldf<bf16>(const bf16* p) { return bf2f(*p); }
template <typename T> DEVINLINE void stf(T* p, float v);
template <> DEVINLINE void stf<float>(float* p, float v) { *p = v; }
template <> DEVINLINE void stf<bf16>(bf16* p, float v) { *p = f2bf(v); }

// one wave: the `top` largest of val(0..E-1), the lower index first among
// equals; lane j receives the j-th chosen value and its index
template <typename F>
DEVINLINE void pick_top(F val, int E, int top, float& mine, int& mine_e) {
  const int lane = threadIdx.x & (WAVE_SIZE - 1);
  unsigned taken = 0;
  mine = 0.f;
  mine_e = 0;
  for (int j = 0; j < top; ++j) {
    float best = -INFINITY;
    int be = 0x7fffffff;
    for (int e = lane, k = 0; e < E; e += WAVE_SIZE, ++k) {
      if (taken & (1u << k)) continue;
      float v = val(e);
      if (!(v > -INFINITY)) v = -INFINITY;       // NaN counts as smallest
      if (v > best || (v == best && e < be)) {
        best = v;
        be = e;
      }
    }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) {
      const float ov = __shfl_xor(best, off, WAVE_SIZE);
      const int oe = __shfl_xor(be, off, WAVE_SIZE);
      if (ov > best || (ov == best && oe < be)) {
        best = ov;
        be = oe;
      }
    }
    if ((be & (WAVE_SIZE - 1)) == lane) taken |= 1u << (be / WAVE_SIZE);
    if (lane == j) {
      mine = best;
      mine_e = be;
    }
  }
}

// the `top` largest logits, weighted by the softmax over the chosen ones
DEVINLINE void select_top(const float* z, int E, int top, float* wt,
                          int* idx) {
  const int lane = threadIdx.x & (WAVE_SIZE - 1);
  float mine;
  int mine_e;
  pick_top([&](int e) { return z[e]; }, E, top, mine, mine_e);
  const float m = __shfl(mine, 0, WAVE_SIZE);    // the largest comes first
  const float ex = lane < top ? expf(mine - m) : 0.f;
  const float tot = wave_reduce_sum(ex);
  if (lane < top) {
    wt[lane] = ex / tot;
    idx[lane] = mine_e;
  }
}

// one block per token: logits, then the selection
template <typename T>
__global__ __launch_bounds__(BLOCK) void route_logits_kernel(
    const T* __restrict__ h, const float* __restrict__ w,
    float* __restrict__ wt, int* __restrict__ idx, int W, int E, int top) {
  extern __shared__ float z[];       // [E]
  const int64_t t = blockIdx.x;
  const int lane = threadIdx.x & (WAVE_SIZE - 1);
  const T* hr = h + t * W;
  for (int e = threadIdx.x / WAVE_SIZE; e < E; e += NWAVE) {
    const float* wr = w + (int64_t)e * W;
    float s = 0.f;
    for (int c = lane; c < W; c += WAVE_SIZE) s += ldf<T>(hr + c) * wr[c];
    s = wave_reduce_sum(s);
    if (lane == 0) z[e] = s;
  }
  __syncthreads();
  if (threadIdx.x < WAVE_SIZE)
    select_top(z, E, top, wt + t * top, idx + t * top);
}

// the same for W a multiple of 4: the token's row is staged in LDS and four
// experts' rows are read side by side, 16 bytes at a time
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

template <typename T>
__global__ __launch_bounds__(BLOCK) void route_logits_vec_kernel(
    const T* __restrict__ h, const float* __restrict__ w,
    float* __restrict__ wt, int* __restrict__ idx, int W, int E, int top) {
  extern __shared__ __align__(16) float sh[];       // hs[W] | z[E]
  float* hs = sh;
  float* z = sh + W;
  const int64_t t = blockIdx.x;
  const int lane = threadIdx.x & (WAVE_SIZE - 1);
  for (int c = threadIdx.x * 4; c < W; c += BLOCK * 4)
    *reinterpret_cast<float4*>(hs + c) = ld4(h + t * W + c);
  __syncthreads();
  for (int e0 = (threadIdx.x / WAVE_SIZE) * 4; e0 < E; e0 += NWAVE * 4) {
    const float* wr[4];
    float s[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int u = 0; u < 4; ++u) wr[u] = w + (int64_t)min(e0 + u, E - 1) * W;
#pragma unroll 4
    for (int c = lane * 4; c < W; c += WAVE_SIZE * 4) {
      const float4 x = *reinterpret_cast<const float4*>(hs + c);
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const float4 y = ld4(wr[u] + c);
        s[u] += x.x * y.x + x.y * y.y + x.z * y.z + x.w * y.w;
      }
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const float v = wave_reduce_sum(s[u]);
      if (lane == 0 && e0 + u < E) z[e0 + u] = v;
    }
  }
  __syncthreads();
  if (threadIdx.x < WAVE_SIZE)
    select_top(z, E, top, wt + t * top, idx + t * top);
}

// one wave per token, logits given (rows of stride ldz): scores s = softmax
// over all experts, chosen by s + corr, weighted by s
__global__ __launch_bounds__(BLOCK) void route_scores_kernel(
    const float* __restrict__ z, int64_t ldz, const float* __restrict__ corr,
    float* __restrict__ wt, int* __restrict__ idx, int64_t T, int E,
    int top) {
  const int64_t t = (int64_t)blockIdx.x * NWAVE + threadIdx.x / WAVE_SIZE;
  if (t >= T) return;
  const int lane = threadIdx.x & (WAVE_SIZE - 1);
  const float* zr = z + t * ldz;
  float m = -INFINITY;
  for (int e = lane; e < E; e += WAVE_SIZE) m = fmaxf(m, zr[e]);
  m = wave_reduce_max(m);
  float sum = 0.f;
  for (int e = lane; e < E; e += WAVE_SIZE) sum += expf(zr[e] - m);
  const float inv = 1.f / wave_reduce_sum(sum);
  float mine;
  int me;
  pick_top([&](int e) { return expf(zr[e] - m) * inv + (corr ? corr[e] : 0.f); },
           E, top, mine, me);
  if (lane < top) {
    me = min(me, E - 1);
    wt[t * top + lane] = expf(zr[me] - m) * inv;
    idx[t * top + lane] = me;
  }
}

// one wave per token, logits given
__global__ __launch_bounds__(BLOCK) void route_select_kernel(
    const float* __restrict__ z, float* __restrict__ wt,
    int* __restrict__ idx, int64_t T, int E, int top) {
  const int64_t t = (int64_t)blockIdx.x * NWAVE + threadIdx.x / WAVE_SIZE;
  if (t >= T) return;
  select_top(z + t * E, E, top, wt + t * top, idx + t * top);
}

// ------------------------------------------------------------------ sort
DEVINLINE void seg_scan(const int* cnt, int* seg, int E) {
  // one thread: E is small and this runs once per step and layer
  int run = 0;
  for (int e = 0; e < E; ++e) {
    seg[e] = run;
    run += cnt[e];
  }
  seg[E] = run;
}

// everything in one block (few pairs): seg [E+1], pair_tok, rank [P]
__global__ __launch_bounds__(BLOCK) void sort_small_kernel(
    const int* __restrict__ idx, int P, int E, int top,
    int* __restrict__ seg, int* __restrict__ pair_tok,
    int* __restrict__ rank) {
  extern __shared__ int ish[];       // cnt[E] | seg[E+1]
  int* cnt = ish;
  int* sg = ish + E;
  for (int e = threadIdx.x; e < E; e += BLOCK) cnt[e] = 0;
  __syncthreads();
  for (int i = threadIdx.x; i < P; i += BLOCK) atomicAdd(&cnt[idx[i]], 1);
  __syncthreads();
  if (threadIdx.x == 0) seg_scan(cnt, sg, E);
  __syncthreads();
  for (int e = threadIdx.x; e <= E; e += BLOCK) seg[e] = sg[e];
  __syncthreads();
  for (int i = threadIdx.x; i < P; i += BLOCK) {
    const int pos = atomicAdd(&sg[idx[i]], 1);
    rank[i] = pos;
    pair_tok[pos] = i / top;
  }
}

__global__ __launch_bounds__(BLOCK) void sort_hist_kernel(
    const int* __restrict__ idx, int P, int E, int* __restrict__ hist) {
  extern __shared__ int ish[];
  for (int e = threadIdx.x; e < E; e += BLOCK) ish[e] = 0;
  __syncthreads();
  const int i1 = min(P, ((int)blockIdx.x + 1) * TILE);
  for (int i = blockIdx.x * TILE + threadIdx.x; i < i1; i += BLOCK)
    atomicAdd(&ish[idx[i]], 1);
  __syncthreads();
  for (int e = threadIdx.x; e < E; e += BLOCK)
    hist[(int64_t)blockIdx.x * E + e] = ish[e];
}

// one block: hist [nb][E] -> each block's first position per expert; seg
__global__ __launch_bounds__(BLOCK) void sort_scan_kernel(
    int* __restrict__ hist, int nb, int E, int* __restrict__ seg) {
  extern __shared__ int ish[];       // cnt[E] | seg[E+1]
  int* cnt = ish;
  int* sg = ish + E;
  for (int e = threadIdx.x; e < E; e += BLOCK) {
    int run = 0;
    for (int k = 0; k < nb; ++k) run += hist[(int64_t)k * E + e];
    cnt[e] = run;
  }
  __syncthreads();
  if (threadIdx.x == 0) seg_scan(cnt, sg, E);
  __syncthreads();
  for (int e = threadIdx.x; e <= E; e += BLOCK) seg[e] = sg[e];
  for (int e = threadIdx.x; e < E; e += BLOCK) {
    int run = sg[e];
    for (int k = 0; k < nb; ++k) {
      const int c = hist[(int64_t)k * E + e];
      hist[(int64_t)k * E + e] = run;
      run += c;
    }
  }
}

__global__ __launch_bounds__(BLOCK) void sort_scatter_kernel(
    const int* __restrict__ idx, int P, int E, int top,
    const int* __restrict__ first, int* __restrict__ pair_tok,
    int* __restrict__ rank) {
  extern __shared__ int ish[];       // next free position per expert
  for (int e = threadIdx.x; e < E; e += BLOCK)
    ish[e] = first[(int64_t)blockIdx.x * E + e];
  __syncthreads();
  const int i1 = min(P, ((int)blockIdx.x + 1) * TILE);
  for (int i = blockIdx.x * TILE + threadIdx.x; i < i1; i += BLOCK) {
    const int pos = atomicAdd(&ish[idx[i]], 1);
    rank[i] = pos;
    pair_tok[pos] = i / top;
  }
}

// --------------------------------------------------------- grouped product
// out[p][n] = sum_k x[tok_idx ? tok_idx[p] : p][k] w[e][n][k] for the pairs p
// of expert e = blockIdx.y; any size, fp32 accumulation in k order
constexpr int GT = 32;               // rows and columns of a tile, k's staged

template <typename T>
__global__ __launch_bounds__(BLOCK) void grouped_any_kernel(
    const T* __restrict__ x, const int* __restrict__ tok_idx,
    const int* __restrict__ seg, const T* __restrict__ w,
    T* __restrict__ out, int N, int K) {
  __shared__ float xs[GT][GT + 1], ws[GT][GT + 1];
  const int e = blockIdx.y, n0 = blockIdx.x * GT;
  const int m0 = seg[e], mt = seg[e + 1] - m0;
  const T* we = w + (int64_t)e * N * K;
  const int tx = threadIdx.x & (GT - 1), ty = threadIdx.x / GT;   // ty < 8
  for (int mb = blockIdx.z * GT; mb < mt; mb += gridDim.z * GT) {
    float acc[4] = {0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < K; k0 += GT) {
      __syncthreads();
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int r = ty + u * 8, k = k0 + tx;
        float xv = 0.f, wv = 0.f;
        if (mb + r < mt && k < K) {
          const int pr = m0 + mb + r;
          xv = ldf<T>(x + (int64_t)(tok_idx ? tok_idx[pr] : pr) * K + k);
        }
        if (n0 + r < N && k < K) wv = ldf<T>(we + (int64_t)(n0 + r) * K + k);
        xs[r][tx] = xv;
        ws[r][tx] = wv;
      }
      __syncthreads();
#pragma unroll
      for (int k = 0; k < GT; ++k) {
        const float wv = ws[tx][k];
#pragma unroll
        for (int u = 0; u < 4; ++u) acc[u] += xs[ty + u * 8][k] * wv;
      }
    }
    if (n0 + tx < N)
#pragma unroll
      for (int u = 0; u < 4; ++u)
        if (mb + ty + u * 8 < mt)
          stf<T>(out + (int64_t)(m0 + mb + ty + u * 8) * N + n0 + tx, acc[u]);
  }
}

// --------------------------------------------------------------- combine
// out[t] = sum_j wt[t][j] y[rank[t][j]] (+ sigmoid(sg[t]) * shared[t]). With
// `ident` [T, W] the pairs at sorted positions >= *n_real belong to identity
// experts, whose output is the token's own row of it.
template <typename T>
__global__ __launch_bounds__(BLOCK) void combine_kernel(
    const T* __restrict__ y, const int* __restrict__ rank,
    const float* __restrict__ wt, const T* __restrict__ shared,
    const T* __restrict__ sg, int ldg, int sg_col,
    const T* __restrict__ ident, const int* __restrict__ n_real,
    T* __restrict__ out, int W, int top) {
  const int64_t t = blockIdx.x;
  const int real = ident ? *n_real : 0x7fffffff;
  float f = 0.f;
  if (shared) {
    f = 1.f;
    if (sg) f = 1.f / (1.f + expf(-ldf<T>(sg + t * ldg + sg_col)));
  }
  for (int c = blockIdx.y * BLOCK + threadIdx.x; c < W;
       c += gridDim.y * BLOCK) {
    float a = 0.f;
    for (int j = 0; j < top; ++j) {
      const int r = rank[t * top + j];
      const T* src = r < real ? y + (int64_t)r * W : ident + t * W;
      a += wt[t * top + j] * ldf<T>(src + c);
    }
    if (shared) a += f * ldf<T>(shared + t * W + c);
    stf<T>(out + t * W + c, a);
  }
}

// bf16 rows of a multiple of 8 columns
__global__ __launch_bounds__(BLOCK) void combine_vec8_kernel(
    const bf16* __restrict__ y, const int* __restrict__ rank,
    const float* __restrict__ wt, const bf16* __restrict__ shared,
    const bf16* __restrict__ sg, int ldg, int sg_col,
    const bf16* __restrict__ ident, const int* __restrict__ n_real,
    bf16* __restrict__ out, int64_t n8, int W, int top) {
  const int W8 = W / 8;
  const int real = ident ? *n_real : 0x7fffffff;
  for (int64_t i = (int64_t)blockIdx.x * BLOCK + threadIdx.x; i < n8;
       i += (int64_t)gridDim.x * BLOCK) {
    const int64_t t = i / W8;
    const int c = (int)(i - t * W8) * 8;
    float a[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    for (int j = 0; j < top; ++j) {
      const float w = wt[t * top + j];
      const int r = rank[t * top + j];
      const bf16* src = r < real ? y + (int64_t)r * W : ident + t * W;
      const bf16x8 v = *reinterpret_cast<const bf16x8*>(src + c);
#pragma unroll
      for (int e = 0; e < 8; ++e) a[e] += w * bf2f(v.v[e]);
    }
    if (shared) {
      const float f =
          sg ? 1.f / (1.f + expf(-bf2f(sg[t * ldg + sg_col]))) : 1.f;
      const bf16x8 v = *reinterpret_cast<const bf16x8*>(shared + t * W + c);
#pragma unroll
      for (int e = 0; e < 8; ++e) a[e] += f * bf2f(v.v[e]);
    }
    bf16x8 o;
#pragma unroll
    for (int e = 0; e < 8; ++e) o.v[e] = f2bf(a[e]);
    *reinterpret_cast<bf16x8*>(out + t * W + c) = o;
  }
}

}  // namespace

extern "C" {

int tl_moe_max_experts() { return MAX_E; }
int tl_moe_max_top() { return MAX_TOP; }

// z null: the logits are computed here (few rows)
void tl_moe_route(const void* h, const void* w, const void* z, void* wt,
                  void* idx, int64_t T, int W, int E, int top, int is_f32,
                  hipStream_t stream) {
  if (T <= 0) return;
  dim3 block(BLOCK);
  if (z) {
    hipLaunchKernelGGL(route_select_kernel,
                       dim3((unsigned)((T + NWAVE - 1) / NWAVE)), block, 0,
                       stream, (const float*)z, (float*)wt, (int*)idx, T, E,
                       top);
    return;
  }
  const size_t smem = sizeof(float) * E;
  dim3 grid((unsigned)T);
  const size_t vmem = sizeof(float) * ((size_t)W + E);
  if (W % 4 == 0 && vmem <= 48 * 1024) {
    if (is_f32)
      hipLaunchKernelGGL(route_logits_vec_kernel<float>, grid, block, vmem,
                         stream, (const float*)h, (const float*)w, (float*)wt,
                         (int*)idx, W, E, top);
    else
      hipLaunchKernelGGL(route_logits_vec_kernel<bf16>, grid, block, vmem,
                         stream, (const bf16*)h, (const float*)w, (float*)wt,
                         (int*)idx, W, E, top);
    return;
  }
  if (is_f32)
    hipLaunchKernelGGL(route_logits_kernel<float>, grid, block, smem, stream,
                       (const float*)h, (const float*)w, (float*)wt,
                       (int*)idx, W, E, top);
  else
    hipLaunchKernelGGL(route_logits_kernel<bf16>, grid, block, smem, stream,
                       (const bf16*)h, (const float*)w, (float*)wt,
                       (int*)idx, W, E, top);
}

// z: first logit of row 0, rows of stride ldz; corr [E] or null
void tl_moe_route_scores(const void* z, int64_t ldz, const void* corr,
                         void* wt, void* idx, int64_t T, int E, int top,
                         hipStream_t stream) {
  if (T <= 0) return;
  hipLaunchKernelGGL(route_scores_kernel,
                     dim3((unsigned)((T + NWAVE - 1) / NWAVE)), dim3(BLOCK), 0,
                     stream, (const float*)z, ldz, (const float*)corr,
                     (float*)wt, (int*)idx, T, E, top);
}

// blocks whose counts the caller's scratch [blocks][E] must hold (0: none)
int tl_moe_sort_blocks(int P) { return P <= TILE ? 0 : (P + TILE - 1) / TILE; }

void tl_moe_sort(const void* idx, int P, int E, int top, void* seg,
                 void* pair_tok, void* rank, void* hist, hipStream_t stream) {
  dim3 block(BLOCK);
  const size_t s1 = sizeof(int) * E, s2 = sizeof(int) * (2 * E + 1);
  const int nb = tl_moe_sort_blocks(P);
  if (nb == 0) {
    hipLaunchKernelGGL(sort_small_kernel, dim3(1), block, s2, stream,
                       (const int*)idx, P, E, top, (int*)seg, (int*)pair_tok,
                       (int*)rank);
    return;
  }
  hipLaunchKernelGGL(sort_hist_kernel, dim3(nb), block, s1, stream,
                     (const int*)idx, P, E, (int*)hist);
  hipLaunchKernelGGL(sort_scan_kernel, dim3(1), block, s2, stream, (int*)hist,
                     nb, E, (int*)seg);
  hipLaunchKernelGGL(sort_scatter_kernel, dim3(nb), block, s1, stream,
                     (const int*)idx, P, E, top, (const int*)hist,
                     (int*)pair_tok, (int*)rank);
}

void tl_grouped_any(const void* x, const void* tok_idx, const void* seg,
                    const void* w, void* out, int P, int E, int N, int K,
                    int is_f32, hipStream_t stream) {
  if (P <= 0) return;
  const int mz = (P + GT - 1) / GT;
  dim3 grid((N + GT - 1) / GT, E, mz < 16 ? mz : 16), block(BLOCK);
  if (is_f32)
    hipLaunchKernelGGL(grouped_any_kernel<float>, grid, block, 0, stream,
                       (const float*)x, (const int*)tok_idx, (const int*)seg,
                       (const float*)w, (float*)out, N, K);
  else
    hipLaunchKernelGGL(grouped_any_kernel<bf16>, grid, block, 0, stream,
                       (const bf16*)x, (const int*)tok_idx, (const int*)seg,
                       (const bf16*)w, (bf16*)out, N, K);
}

void tl_moe_combine(const void* y, const void* rank, const void* wt,
                    const void* shared, const void* sg, int ldg, int sg_col,
                    const void* ident, const void* n_real, void* out,
                    int64_t T, int W, int top, int is_f32,
                    hipStream_t stream) {
  if (T <= 0) return;
  if (!is_f32 && W % 8 == 0) {
    const int64_t n8 = T * (W / 8);
    const int64_t nb = (n8 + BLOCK - 1) / BLOCK;
    hipLaunchKernelGGL(combine_vec8_kernel,
                       dim3((unsigned)(nb > 8192 ? 8192 : nb)), dim3(BLOCK), 0,
                       stream, (const bf16*)y, (const int*)rank,
                       (const float*)wt, (const bf16*)shared, (const bf16*)sg,
                       ldg, sg_col, (const bf16*)ident, (const int*)n_real,
                       (bf16*)out, n8, W, top);
    return;
  }
  const int cb = (W + BLOCK - 1) / BLOCK;
  dim3 grid((unsigned)T, cb < 8 ? cb : 8), block(BLOCK);
  if (is_f32)
    hipLaunchKernelGGL(combine_kernel<float>, grid, block, 0, stream,
                       (const float*)y, (const int*)rank, (const float*)wt,
                       (const float*)shared, (const float*)sg, ldg, sg_col,
                       (const float*)ident, (const int*)n_real, (float*)out,
                       W, top);
  else
    hipLaunchKernelGGL(combine_kernel<bf16>, grid, block, 0, stream,
                       (const bf16*)y, (const int*)rank, (const float*)wt,
                       (const bf16*)shared, (const bf16*)sg, ldg, sg_col,
                       (const bf16*)ident, (const int*)n_real, (bf16*)out, W,
                       top);
}

}  // extern "C"
