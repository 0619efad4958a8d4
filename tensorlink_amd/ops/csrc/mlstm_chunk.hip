// Matrix-memory (mLSTM) recurrence for long prompt portions: chunk form on
// the fp32 MFMA (gfx950). The recurrence, its state and the fused read-out
// (per-head unit RMS, norm weight, sigmoid gate) are those of mlstm_scan.hip.
//
// A sequence's tokens are cut into chunks of 64. Inside a chunk, with F_t
// the running sum of log forget gates, a_s = i_s - F_s and m0 the running
// maximum before the chunk,
//     M_t = max(m0, max_{s<=t} a_s),   m_t = F_t + M_t
//     num_t = sum_{s<=t} e^(a_s - M_t) (q_t . k_s) v_s + e^(m0 - M_t) S0^T q_t
//     n_t . q_t likewise with v = 1 and n0
//     S1 = e^(m0 - M_C) S0 + sum_s e^(a_s - M_C) k_s v_s^T
// Every exponent is <= 0. F and a are kept in double, so that their
// differences are as exact as token by token.
//
// tl_mlstm_chunks runs four kernels: every chunk's own contribution with its
// own maximum A = max a (state_kernel); the chain of maxima and factors, one
// wave per (sequence, head) (scale_kernel); the elementwise chain over the
// states, which replaces a chunk's contribution by the state before it
// (chain_kernel); the read-outs, one block per (chunk, head), one wave per
// 16 tokens, a wave holding whole rows of V so that the norm and the gate
// are applied in registers (out_kernel).
//
// MFMA operands (16x16x4): lane (i = lane & 15, g = lane >> 4) supplies A[i][k]
// and B[k][i] of one k per instruction and receives rows 4g .. 4g + 3 of
// column i. The order of the k's is free: group g takes k = 4g + s at step s.
// The scores are computed transposed (keys as rows), so their accumulator is
// the A operand of the product with the values as it stands. Column i of value
// tile n is column 64 (n / 4) + 4 i + n % 4 of memory: a lane's columns come
// in fours, and the fours of neighbouring lanes are contiguous.

#include "common.hpp"

namespace {

constexpr int BLOCK = 256;
constexpr int C = 64;                // tokens per chunk

using f32x4 = __attribute__((ext_vector_type(4))) float;

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
DEVINLINE void st4(float* p, const float (&v)[4]) {
  *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
}
DEVINLINE void st4(bf16* p, const float (&v)[4]) {
  bf16x4 o;
#pragma unroll
  for (int e = 0; e < 4; ++e) o.v[e] = f2bf(v[e]);
  *reinterpret_cast<bf16x4*>(p) = o;
}

DEVINLINE float log_sigmoid(float x) {
  return fminf(x, 0.f) - log1pf(expf(-fabsf(x)));
}

struct MlSrc {
  int ld, q_off, k_off, v_off, g_off;
  const float* gates;      // raw input | forget pre-activations
  int ldg;
  float cap, qscale, eps;
};

// first wave: F[t], a[t] of the chunk's n tokens (a = -inf beyond)
DEVINLINE void chunk_gates(const MlSrc& p, int t0, int n, int h, int H,
                           double* F, double* a) {
  const int t = threadIdx.x;
  if (t >= C) return;
  double f = 0.0, li = 0.0;
  if (t < n) {
    const float* g = p.gates + (int64_t)(t0 + t) * p.ldg;
    li = (double)(p.cap * tanhf(g[h] / p.cap));
    f = (double)log_sigmoid(p.cap * tanhf(g[H + h] / p.cap));
  }
#pragma unroll
  for (int off = 1; off < C; off <<= 1) {
    const double o = __shfl_up(f, off, WAVE_SIZE);
    if (t >= off) f += o;
  }
  F[t] = f;
  a[t] = t < n ? li - f : -INFINITY;
}

// a lane's NV columns from c; columns beyond V (a multiple of 4) read as 0. Loads are
// unconditional, from the nearest place that exists: no branch around a load,
// so that many are in flight together.
template <int NV, typename T>
DEVINLINE void ld_cols(const T* row, int c, int V, float (&o)[NV]) {
#pragma unroll
  for (int n = 0; n < NV; n += 4) {
    float x[4];
    ld4(row + min(c + n * 16, V - 4), x);
#pragma unroll
    for (int e = 0; e < 4; ++e) o[n + e] = c + n * 16 < V ? x[e] : 0.f;
  }
}

// grid (chunks, H)
template <typename T, int NV>
__global__ __launch_bounds__(BLOCK) void mlstm_state_kernel(
    const T* __restrict__ proj, MlSrc p, const int* __restrict__ cu_c,
    float* __restrict__ U, float* __restrict__ nU, float* __restrict__ Amax,
    float* __restrict__ Fsum, int H, int D, int V) {
  __shared__ double F[C], a[C];
  __shared__ float w[C];
  const int ch = blockIdx.x, h = blockIdx.y;
  const int t0 = cu_c[ch], n = cu_c[ch + 1] - t0;
  const int64_t ci = (int64_t)ch * H + h;
  chunk_gates(p, t0, n, h, H, F, a);
  if (threadIdx.x < C) {
    double m = a[threadIdx.x];
#pragma unroll
    for (int off = 32; off > 0; off >>= 1)
      m = fmax(m, __shfl_xor(m, off, WAVE_SIZE));
    // the stored maximum is the rounded one; the weights use it as it is
    const float mf = (float)m;
    w[threadIdx.x] = expf((float)(a[threadIdx.x] - (double)mf));
    if (threadIdx.x == 0) {
      Amax[ci] = mf;
      Fsum[ci] = (float)F[C - 1];
    }
  }
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int li = lane & 15, quad = lane >> 4;
  const int nd = (D + 15) / 16, nv = (V + 16 * NV - 1) / (16 * NV);
  float* Uc = U + ci * D * V;
  for (int u = wave; u < nd * nv; u += 4) {
    const int d0 = (u % nd) * 16, c = (u / nd) * 16 * NV + li * 4;
    f32x4 acc[NV];
#pragma unroll
    for (int x = 0; x < NV; ++x) acc[x] = (f32x4){0.f, 0.f, 0.f, 0.f};
    float ns = 0.f;
    const bool din = d0 + li < D;
#pragma unroll 4
    for (int s = 0; s < C / 4; ++s) {
      const int j = quad * (C / 4) + s;
      const T* row = proj + (int64_t)(t0 + min(j, n - 1)) * p.ld;
      float kw, vv[NV];
      if constexpr (sizeof(T) == 2)
        kw = bf2f(row[p.k_off + h * D + min(d0 + li, D - 1)]);
      else
        kw = row[p.k_off + h * D + min(d0 + li, D - 1)];
      kw = din ? kw * w[j] : 0.f;    // w is 0 beyond the chunk's tokens
      ld_cols<NV, T>(row + p.v_off + h * V, c, V, vv);
      ns += kw;
#pragma unroll
      for (int x = 0; x < NV; ++x)
        acc[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(kw, vv[x], acc[x], 0, 0,
                                                      0);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = d0 + quad * 4 + r;
      if (d >= D) continue;
#pragma unroll
      for (int x = 0; x < NV; x += 4)
        if (c + x * 16 < V) {
          const float o[4] = {acc[x][r], acc[x + 1][r], acc[x + 2][r],
                              acc[x + 3][r]};
          st4(Uc + (int64_t)d * V + c + x * 16, o);
        }
    }
    if (u < nd) {                    // the same with v = 1
      ns += __shfl_xor(ns, 16, WAVE_SIZE);
      ns += __shfl_xor(ns, 32, WAVE_SIZE);
      if (quad == 0 && din) nU[ci * D + d0 + li] = ns;
    }
  }
}

// one wave per (sequence, head): per chunk the factors of the state before
// (ca) and of the chunk's contribution (cb), and the maximum before it (mb)
__global__ __launch_bounds__(WAVE_SIZE) void mlstm_scale_kernel(
    const float* __restrict__ Amax, const float* __restrict__ Fsum,
    float* __restrict__ ca, float* __restrict__ cb, float* __restrict__ mb,
    float* __restrict__ m_pool, const int* __restrict__ chunk_base,
    const int* __restrict__ n_chunks, const int* __restrict__ slots,
    const int* __restrict__ pos0, int H) {
  const int b = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const int c0 = chunk_base[b], nc = n_chunks[b];
  if (nc <= 0) return;
  float* mp = m_pool + (int64_t)slots[b] * H + h;
  float m = pos0[b] == 0 ? 0.f : *mp;
  for (int k0 = 0; k0 < nc; k0 += WAVE_SIZE) {
    const int k = k0 + lane;
    const int64_t ci = (int64_t)(c0 + k) * H + h;
    float A = 0.f, F = 0.f, before = 0.f, top = 0.f;
    if (k < nc) {
      A = Amax[ci];
      F = Fsum[ci];
    }
    const int cnt = min(WAVE_SIZE, nc - k0);
    for (int i = 0; i < cnt; ++i) {
      const float Ai = __shfl(A, i, WAVE_SIZE), Fi = __shfl(F, i, WAVE_SIZE);
      const float M = fmaxf(m, Ai);
      if (lane == i) {
        before = m;
        top = M;
      }
      m = Fi + M;
    }
    if (k < nc) {
      ca[ci] = expf(before - top);
      cb[ci] = expf(A - top);
      mb[ci] = before;
    }
  }
  if (lane == 0) *mp = m;
}

// grid (B, H, ceil((D*V + D) / BLOCK)): U and nU hold the chunks' own
// contributions on entry and the state before each chunk on exit; the slot
// receives the state after the last one
__global__ __launch_bounds__(BLOCK) void mlstm_chain_elem_kernel(
    float* __restrict__ U, float* __restrict__ nU,
    const float* __restrict__ ca, const float* __restrict__ cb,
    float* __restrict__ S, float* __restrict__ n,
    const int* __restrict__ chunk_base, const int* __restrict__ n_chunks,
    const int* __restrict__ slots, const int* __restrict__ pos0, int H,
    int D, int DV) {
  const int b = blockIdx.x, h = blockIdx.y;
  int e = blockIdx.z * BLOCK + threadIdx.x;
  const int nc = n_chunks[b];
  if (e >= DV + D || nc <= 0) return;
  const bool isS = e < DV;
  if (!isS) e -= DV;
  const int E = isS ? DV : D;
  float* pool = (isS ? S : n) + ((int64_t)slots[b] * H + h) * E + e;
  float* up = (isS ? U : nU) + ((int64_t)chunk_base[b] * H + h) * E + e;
  const int64_t su = (int64_t)H * E;
  const float* ap = ca + (int64_t)chunk_base[b] * H + h;
  const float* bp = cb + (int64_t)chunk_base[b] * H + h;
  float s = pos0[b] == 0 ? 0.f : *pool;
  int c = 0;
  for (; c + 4 <= nc; c += 4) {      // four chunks are loaded ahead of use
    float u[4], fa[4], fb[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      u[i] = up[i * su];
      fa[i] = ap[i * H];
      fb[i] = bp[i * H];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      up[i * su] = s;
      s = fa[i] * s + fb[i] * u[i];
    }
    up += 4 * su;
    ap += 4 * H;
    bp += 4 * H;
  }
  for (; c < nc; ++c) {
    const float u = *up;
    *up = s;
    s = *ap * s + *bp * u;
    up += su;
    ap += H;
    bp += H;
  }
  *pool = s;
}

// grid (chunks, H): wave w reads out tokens 16w .. 16w + 15
template <typename T, int DT, int NV>
__global__ __launch_bounds__(BLOCK) void mlstm_out_kernel(
    const T* __restrict__ proj, MlSrc p, const int* __restrict__ cu_c,
    const float* __restrict__ U, const float* __restrict__ nU,
    const float* __restrict__ mb, const float* __restrict__ norm_w,
    T* __restrict__ out, int H, int D, int V) {
  __shared__ double F[C], a[C], M[C];
  const int ch = blockIdx.x, h = blockIdx.y;
  const int t0 = cu_c[ch], n = cu_c[ch + 1] - t0;
  const int64_t ci = (int64_t)ch * H + h;
  const float m0 = mb[ci];
  chunk_gates(p, t0, n, h, H, F, a);
  if (threadIdx.x < C) {             // running maximum
    double m = fmax(a[threadIdx.x], (double)m0);
#pragma unroll
    for (int off = 1; off < C; off <<= 1) {
      const double o = __shfl_up(m, off, WAVE_SIZE);
      if (threadIdx.x >= off) m = fmax(m, o);
    }
    M[threadIdx.x] = m;
  }
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int li = lane & 15, quad = lane >> 4;
  if (wave * 16 >= n) return;        // no barrier below
  const int t = wave * 16 + li;      // this lane's query
  const int c = li * 4;              // and its first value column
  const T* kh = proj + (int64_t)t0 * p.ld + p.k_off + h * D;
  const T* vh = proj + (int64_t)t0 * p.ld + p.v_off + h * V;
  const double Mt = M[t];
  const float carry = expf((float)((double)m0 - Mt));
  float q[DT][4];
  float nq = 0.f;
  const float* n0 = nU + ci * D;
#pragma unroll
  for (int dt = 0; dt < DT; ++dt) {
    const int d = dt * 16 + quad * 4, dc = min(d, D - 4);
    float x[4], y[4];
    ld4(proj + (int64_t)(t0 + min(t, n - 1)) * p.ld + p.q_off + h * D + dc, x);
    ld4(n0 + dc, y);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      q[dt][e] = d < D && t < n ? x[e] * p.qscale : 0.f;
      nq += q[dt][e] * y[e];
    }
  }
  nq *= carry;
  f32x4 acc[NV];
#pragma unroll
  for (int x = 0; x < NV; ++x) acc[x] = (f32x4){0.f, 0.f, 0.f, 0.f};
  // the carried part
  const float* Uc = U + ci * D * V;
#pragma unroll
  for (int dt = 0; dt < DT; ++dt) {
    if (dt * 16 < D) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int d = dt * 16 + quad * 4 + e;
        float s0[NV];                // (q is 0 beyond D)
        ld_cols<NV, float>(Uc + (int64_t)min(d, D - 1) * V, c, V, s0);
        const float qe = q[dt][e] * carry;
#pragma unroll
        for (int x = 0; x < NV; ++x)
          acc[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(qe, s0[x], acc[x], 0,
                                                        0, 0);
      }
    }
  }
  // the chunk's own part, 16 keys at a time
  for (int b = 0; b <= wave; ++b) {
    f32x4 sc = (f32x4){0.f, 0.f, 0.f, 0.f};
    const int j = b * 16 + li;       // this lane's key row
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      float x[4];                    // (q is 0 beyond D, rows beyond n masked)
      ld4(kh + (int64_t)min(j, n - 1) * p.ld +
              min(dt * 16 + quad * 4, D - 4), x);
#pragma unroll
      for (int e = 0; e < 4; ++e)
        sc = __builtin_amdgcn_mfma_f32_16x16x4f32(x[e], q[dt][e], sc, 0, 0, 0);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int s = b * 16 + quad * 4 + e;
      const float w = s <= t && s < n ? sc[e] * expf((float)(a[s] - Mt)) : 0.f;
      nq += w;
      float vv[NV];
      ld_cols<NV, T>(vh + (int64_t)min(s, n - 1) * p.ld, c, V, vv);
#pragma unroll
      for (int x = 0; x < NV; ++x)
        acc[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(w, vv[x], acc[x], 0, 0,
                                                      0);
    }
  }
  nq += __shfl_xor(nq, 16, WAVE_SIZE);
  nq += __shfl_xor(nq, 32, WAVE_SIZE);
  // this lane's query's normaliser; rows of the accumulator fetch theirs
  const float den =
      fmaxf(fabsf(nq), expf((float)(-(F[t] + Mt)))) + 1e-6f;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int tr = wave * 16 + quad * 4 + r;
    const float inv = 1.f / __shfl(den, quad * 4 + r, WAVE_SIZE);
    float ss = 0.f;
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const float o = acc[x][r] * inv;
      acc[x][r] = o;
      ss += o * o;                   // columns beyond V are 0
    }
#pragma unroll
    for (int off = 8; off > 0; off >>= 1) ss += __shfl_xor(ss, off, WAVE_SIZE);
    const float rn = rsqrtf(ss / (float)V + p.eps);
    if (tr < n) {
      const int64_t row = t0 + tr;
      const T* gr = proj + row * p.ld + p.g_off + h * V;
      T* orow = out + (row * H + h) * V;
#pragma unroll
      for (int x = 0; x < NV; x += 4)
        if (c + x * 16 < V) {
          float g[4], w4[4], o[4];
          ld4(gr + c + x * 16, g);
          ld4(norm_w + h * V + c + x * 16, w4);
#pragma unroll
          for (int e = 0; e < 4; ++e)
            o[e] = acc[x + e][r] * rn * w4[e] / (1.f + expf(-g[e]));
          st4(orow + c + x * 16, o);
        }
    }
  }
}

template <typename T>
void launch(const T* proj, const MlSrc& p, const float* norm_w, float* S,
            float* n, float* m, float* U, float* nU, float* sc,
            const int* cu_c, int NC, const int* base, const int* cnt,
            const int* slots, const int* pos0, int B, T* out, int H, int D,
            int V, hipStream_t stream) {
  // sc: Amax | Fsum | ca | cb | mb, [NC * H] each
  const int64_t nh = (int64_t)NC * H;
  float *A = sc, *F = sc + nh, *ca = sc + 2 * nh, *cb = sc + 3 * nh,
        *mb = sc + 4 * nh;
  dim3 grid(NC, H), block(BLOCK);
  if (V <= 64)
    hipLaunchKernelGGL((mlstm_state_kernel<T, 4>), grid, block, 0, stream,
                       proj, p, cu_c, U, nU, A, F, H, D, V);
  else
    hipLaunchKernelGGL((mlstm_state_kernel<T, 8>), grid, block, 0, stream,
                       proj, p, cu_c, U, nU, A, F, H, D, V);
  hipLaunchKernelGGL(mlstm_scale_kernel, dim3(B, H), dim3(WAVE_SIZE), 0,
                     stream, A, F, ca, cb, mb, m, base, cnt, slots, pos0, H);
  hipLaunchKernelGGL(mlstm_chain_elem_kernel,
                     dim3(B, H, (D * V + D + BLOCK - 1) / BLOCK), block, 0,
                     stream, U, nU, ca, cb, S, n, base, cnt, slots, pos0, H, D,
                     D * V);
#define TL_MC(DT, NV)                                                       \
  hipLaunchKernelGGL((mlstm_out_kernel<T, DT, NV>), grid, block, 0, stream, \
                     proj, p, cu_c, (const float*)U, (const float*)nU,      \
                     (const float*)mb, norm_w, out, H, D, V)
#define TL_MC_V(DT)                  \
  if (V <= 64) TL_MC(DT, 4);         \
  else if (V <= 128) TL_MC(DT, 8);   \
  else TL_MC(DT, 16)
  if (D <= 64) { TL_MC_V(4); }
  else if (D <= 128) { TL_MC_V(8); }
  else { TL_MC_V(16); }
#undef TL_MC_V
#undef TL_MC
}

}  // namespace

extern "C" {

int tl_mlstm_chunk_tokens() { return C; }

// 1 if the chunk form serves the shape (sizes, row stride and column offsets
// multiples of 4)
int tl_mlstm_chunks_ok(int D, int V, int ld, int q_off, int k_off, int v_off,
                       int g_off) {
  if (D < 4 || D > 256 || V < 4 || V > 256) return 0;
  return (D | V | ld | q_off | k_off | v_off | g_off) % 4 == 0 ? 1 : 0;
}

// U [NC, H, D, V], nU [NC, H, D], sc [5, NC, H]: fp32 scratch
int tl_mlstm_chunks(const void* proj, int ld, int q_off, int k_off,
                    int v_off, int g_off, const void* gates, int ldg,
                    const void* norm_w, void* S, void* n, void* m, void* U,
                    void* nU, void* sc, const void* cu_c, int NC,
                    const void* base, const void* cnt, const void* slots,
                    const void* pos0, int B, void* out, int H, int D, int V,
                    float cap, float qscale, float eps, int is_f32,
                    hipStream_t stream) {
  if (!tl_mlstm_chunks_ok(D, V, ld, q_off, k_off, v_off, g_off) || H < 1)
    return 1;
  if (NC <= 0 || B <= 0) return 0;
  MlSrc p{ld, q_off, k_off, v_off, g_off, (const float*)gates, ldg, cap,
          qscale, eps};
  if (is_f32)
    launch<float>((const float*)proj, p, (const float*)norm_w, (float*)S,
                  (float*)n, (float*)m, (float*)U, (float*)nU, (float*)sc,
                  (const int*)cu_c, NC, (const int*)base, (const int*)cnt,
                  (const int*)slots, (const int*)pos0, B, (float*)out, H, D,
                  V, stream);
  else
    launch<bf16>((const bf16*)proj, p, (const float*)norm_w, (float*)S,
                 (float*)n, (float*)m, (float*)U, (float*)nU, (float*)sc,
                 (const int*)cu_c, NC, (const int*)base, (const int*)cnt,
                 (const int*)slots, (const int*)pos0, B, (bf16*)out, H, D, V,
                 stream);
  return 0;
}

}  // extern "C"
