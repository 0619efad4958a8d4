// Gated linear attention (one decay per key channel and token) over ragged
// sequences (gfx950).
//
// Per head, q scaled by D^-1/2:
//     z_t = r_t A2 + b,  log alpha_t = log sigmoid(z_t) / tau     [D]
//     S_t = diag(alpha_t) S_(t-1) + k_t v_t^T     (S is [D, V], fp32, per slot)
//     o_t = S_t^T q_t
// q, k, v and the low-rank r are columns of the fused projection (bf16 or
// fp32); everything behind them is fp32. The second factor of the decay's
// projection is applied here, so the decays never make a trip to memory.
//
// tl_gla_scan walks the tokens in order (decoding, short portions). One
// block per (sequence, head, 64 value columns): columns of S are
// independent, so a decode step spreads over B * H * V/64 blocks. Thread
// (c, g) owns column c of S for DR consecutive rows starting at g * DR; a
// token's q, k and decays are read from LDS as broadcast vectors and the
// four partial read-outs of a column meet in LDS. Key sizes beyond the
// register budget take the generic kernel (state in the slot's memory).
//
// Long prompt portions take the chunk form: chunks of C = 16 * NS tokens,
// cut into NS tiles of 16. With l_i the running sum of log alpha INSIDE a
// token's own tile (l_i <= 0) and tot_a the sum over tile a:
//   tile (a, b), b < a:  A_ij = sum_d [q_i e^(l_i + sum_{b<c<a} tot_c)]
//                                     [k_j e^(tot_b - l_j)]
//   diagonal tile:       A_ij = sum_d q_i k_j e^(l_i - l_j),  j <= i
//   o_i = sum_j A_ij v_j + sum_d [q_i e^(l_i + sum_{c<a} tot_c)] S0_d
//   S1  = e^(sum tot) S0 + sum_j [k_j e^(tot_b - l_j + sum_{c>b} tot_c)] v_j^T
// Every exponent of the off-diagonal tiles and of the carried parts is <= 0,
// so nothing overflows however strong the decay. Diagonal tiles factor as
// [q_i e^(l_i)] [k_j e^(-l_j)] when the tile's decay stays within
// LOG_RANGE (then both factors are ordinary fp32 numbers); otherwise the
// 16 x 16 scores are summed with e^(l_i - l_j) directly. All products run on
// the fp32 MFMA (16x16x4). tl_gla_chunk_state writes every chunk's own
// contribution to S1 and its decay, tl_gla_chain turns them into the state
// before each chunk (and leaves the last state in the slot),
// tl_gla_chunk_out computes A and the outputs.
//
// MFMA operands: lane (i = lane & 15, g = lane >> 4) supplies A[i][k] and
// B[k][i] of one k per instruction. The order of the k's is free, so group g
// takes a contiguous stretch of them and loads it as vectors; likewise
// column n of the value tile is mapped to column i * NV + n of memory, so a
// lane's NV columns are contiguous.

#include "common.hpp"

namespace {

constexpr int BLOCK = 256;
constexpr int RT = 8;               // tokens per round of the scan
constexpr int VT = 64;              // value columns per block of the scan
constexpr float LOG_RANGE = 60.f;   // e^60 * e^60 is inside fp32

using f32x4 = __attribute__((ext_vector_type(4))) float;

template <typename T> DEVINLINE float ldf(const T* p);
template <> DEVINLINE float ldf<float>(const float* p) { return *p; }
template <> DEVINLINE float ldf<bf16>(const bf16* p) { return bf2f(*p); }

struct alignas(8) bf16x4 {
  bf16 v[4];
};

// four consecutive elements; `n` of them exist (the rest reads as 0)
template <typename T, bool VEC>
DEVINLINE void ld4(const T* p, int n, float (&o)[4]) {
  if (VEC && n >= 4) {
    if constexpr (sizeof(T) == 2) {
      const bf16x4 x = *reinterpret_cast<const bf16x4*>(p);
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] = bf2f(x.v[e]);
    } else {
      const float4 x = *reinterpret_cast<const float4*>(p);
      o[0] = x.x;
      o[1] = x.y;
      o[2] = x.z;
      o[3] = x.w;
    }
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] = e < n ? ldf<T>(p + e) : 0.f;
  }
}

// log sigmoid(z)
DEVINLINE float log_sigmoid(float z) {
  return fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
}

struct GlaSrc {
  int ld, q_off, k_off, v_off, r_off;
  const float* a2t;    // [R][H*D]
  const float* bias;   // [H*D]
  int R;
  float inv_tau, qscale;
};

// ------------------------------------------------------------------ scan
template <typename T, int DR>
__global__ __launch_bounds__(BLOCK) void gla_scan_kernel(
    const T* __restrict__ proj, GlaSrc p, float* __restrict__ S,
    const int* __restrict__ cu, const int* __restrict__ slots,
    const int* __restrict__ pos0, float* __restrict__ out, int H, int D,
    int V) {
  constexpr int DP = 4 * DR;        // rows of a staged vector
  extern __shared__ __align__(16) float lds[];
  // lds: qs | ks | as [RT][DP] | vs[RT][VT] | part[RT][4][VT] | rs[RT][R]
  float* qs = lds;
  float* ks = qs + RT * DP;
  float* as = ks + RT * DP;
  float* vs = as + RT * DP;
  float* part = vs + RT * VT;
  float* rs = part + RT * 4 * VT;
  const int b = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * VT;
  const int t0 = cu[b], t1 = cu[b + 1];
  if (t1 <= t0) return;
  const int cl = threadIdx.x & (VT - 1), g = threadIdx.x / VT;
  const int c = c0 + cl;
  float* Sh = S + ((int64_t)slots[b] * H + h) * D * V;
  const bool fresh = pos0[b] == 0;
  float st[DR];
#pragma unroll
  for (int r = 0; r < DR; ++r) {
    const int d = g * DR + r;
    st[r] = (!fresh && d < D && c < V) ? Sh[(int64_t)d * V + c] : 0.f;
  }
  for (int tb = t0; tb < t1; tb += RT) {
    const int nt = min(RT, t1 - tb);
    __syncthreads();
    for (int i = threadIdx.x; i < nt * p.R; i += BLOCK) {
      const int tt = i / p.R, r = i - tt * p.R;
      rs[i] = ldf<T>(proj + (int64_t)(tb + tt) * p.ld + p.r_off + r);
    }
    for (int i = threadIdx.x; i < nt * VT; i += BLOCK) {
      const int tt = i / VT, e = i & (VT - 1);
      vs[i] = c0 + e < V ? ldf<T>(proj + (int64_t)(tb + tt) * p.ld + p.v_off +
                                  h * V + c0 + e)
                         : 0.f;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < nt * DP; i += BLOCK) {
      const int tt = i / DP, d = i - tt * DP;
      float q = 0.f, k = 0.f, a = 1.f;
      if (d < D) {
        const int hd = h * D + d;
        const T* row = proj + (int64_t)(tb + tt) * p.ld;
        q = ldf<T>(row + p.q_off + hd) * p.qscale;
        k = ldf<T>(row + p.k_off + hd);
        float z = p.bias[hd];
        for (int r = 0; r < p.R; ++r)
          z += rs[tt * p.R + r] * p.a2t[(int64_t)r * H * D + hd];
        a = expf(log_sigmoid(z) * p.inv_tau);
      }
      qs[i] = q;
      ks[i] = k;
      as[i] = a;
    }
    __syncthreads();
    for (int tt = 0; tt < nt; ++tt) {
      const float vv = vs[tt * VT + cl];
      const float4* a4 = reinterpret_cast<const float4*>(as + tt * DP + g * DR);
      const float4* k4 = reinterpret_cast<const float4*>(ks + tt * DP + g * DR);
      const float4* q4 = reinterpret_cast<const float4*>(qs + tt * DP + g * DR);
      float acc = 0.f;
#pragma unroll
      for (int r = 0; r < DR / 4; ++r) {
        const float4 a = a4[r], k = k4[r], q = q4[r];
        st[4 * r + 0] = a.x * st[4 * r + 0] + k.x * vv;
        st[4 * r + 1] = a.y * st[4 * r + 1] + k.y * vv;
        st[4 * r + 2] = a.z * st[4 * r + 2] + k.z * vv;
        st[4 * r + 3] = a.w * st[4 * r + 3] + k.w * vv;
        acc += st[4 * r + 0] * q.x + st[4 * r + 1] * q.y +
               st[4 * r + 2] * q.z + st[4 * r + 3] * q.w;
      }
      part[(tt * 4 + g) * VT + cl] = acc;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < nt * VT; i += BLOCK) {
      const int tt = i / VT, e = i & (VT - 1);
      if (c0 + e < V) {
        float o = 0.f;
#pragma unroll
        for (int gg = 0; gg < 4; ++gg) o += part[(tt * 4 + gg) * VT + e];
        out[((int64_t)(tb + tt) * H + h) * V + c0 + e] = o;
      }
    }
  }
#pragma unroll
  for (int r = 0; r < DR; ++r) {
    const int d = g * DR + r;
    if (d < D && c < V) Sh[(int64_t)d * V + c] = st[r];
  }
}

// Any key size: the state stays in the slot's memory; thread c owns the
// columns c, c + BLOCK, ... and walks all rows for every token.
template <typename T>
__global__ __launch_bounds__(BLOCK) void gla_scan_generic_kernel(
    const T* __restrict__ proj, GlaSrc p, float* __restrict__ S,
    const int* __restrict__ cu, const int* __restrict__ slots,
    const int* __restrict__ pos0, float* __restrict__ out, int H, int D,
    int V) {
  extern __shared__ __align__(16) float lds[];  // as[D] | ks[D] | qs[D]
  float* as = lds;
  float* ks = as + D;
  float* qs = ks + D;
  const int b = blockIdx.x, h = blockIdx.y;
  const int t0 = cu[b], t1 = cu[b + 1];
  if (t1 <= t0) return;
  float* Sh = S + ((int64_t)slots[b] * H + h) * D * V;
  if (pos0[b] == 0)
    for (int i = threadIdx.x; i < D * V; i += BLOCK) Sh[i] = 0.f;
  for (int t = t0; t < t1; ++t) {
    __syncthreads();
    const T* row = proj + (int64_t)t * p.ld;
    for (int d = threadIdx.x; d < D; d += BLOCK) {
      const int hd = h * D + d;
      qs[d] = ldf<T>(row + p.q_off + hd) * p.qscale;
      ks[d] = ldf<T>(row + p.k_off + hd);
      float z = p.bias[hd];
      for (int r = 0; r < p.R; ++r)
        z += ldf<T>(row + p.r_off + r) * p.a2t[(int64_t)r * H * D + hd];
      as[d] = expf(log_sigmoid(z) * p.inv_tau);
    }
    __syncthreads();
    for (int c = threadIdx.x; c < V; c += BLOCK) {
      const float vv = ldf<T>(row + p.v_off + h * V + c);
      float acc = 0.f;
      for (int d = 0; d < D; ++d) {
        const float s = as[d] * Sh[(int64_t)d * V + c] + ks[d] * vv;
        Sh[(int64_t)d * V + c] = s;
        acc += s * qs[d];
      }
      out[((int64_t)t * H + h) * V + c] = acc;
    }
  }
}

// ----------------------------------------------------------- chunk form
// contiguous k's per lane group of the key dimension, and the LDS row
// stride of [token][channel] arrays (rows start 4 banks apart)
__host__ __device__ inline int quarter(int D) { return (D + 15) / 16 * 4; }
__host__ __device__ inline int row_stride(int D) { return 4 * quarter(D) + 4; }

// L[C][ls]: running sums of log alpha inside each 16-token tile; tot[NS][ls]:
// their last values. Channels beyond D and tokens beyond n add nothing.
// rs[R][C] is scratch; far[a] is set when tile a leaves LOG_RANGE.
template <typename T, int NS>
DEVINLINE void chunk_logs(const T* proj, const GlaSrc& p, int t0, int n,
                          int h, int H, int D, int ls, float* L, float* tot,
                          float* rs, int* far) {
  constexpr int C = 16 * NS;
  if (threadIdx.x < NS) far[threadIdx.x] = 0;
  for (int i = threadIdx.x; i < C * p.R; i += BLOCK) {
    const int t = i / p.R, r = i - t * p.R;
    rs[r * C + t] =
        t < n ? ldf<T>(proj + (int64_t)(t0 + t) * p.ld + p.r_off + r) : 0.f;
  }
  __syncthreads();
  const int DP = ls - 4;
  for (int i = threadIdx.x; i < NS * DP; i += BLOCK) {
    const int a = i / DP, d = i - a * DP;
    float z[16];
    const int hd = h * D + d;
    const float bz = d < D ? p.bias[hd] : 0.f;
#pragma unroll
    for (int t = 0; t < 16; ++t) z[t] = bz;
    if (d < D)
      for (int r = 0; r < p.R; ++r) {
        const float w = p.a2t[(int64_t)r * H * D + hd];
        const float4* rr = reinterpret_cast<const float4*>(rs + r * C + a * 16);
#pragma unroll
        for (int t4 = 0; t4 < 4; ++t4) {
          const float4 x = rr[t4];
          z[4 * t4 + 0] += w * x.x;
          z[4 * t4 + 1] += w * x.y;
          z[4 * t4 + 2] += w * x.z;
          z[4 * t4 + 3] += w * x.w;
        }
      }
    float run = 0.f;
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      if (d < D && a * 16 + t < n) run += log_sigmoid(z[t]) * p.inv_tau;
      L[(a * 16 + t) * ls + d] = run;
    }
    tot[a * ls + d] = run;
    if (run < -LOG_RANGE) far[a] = 1;      // same value from every writer
  }
  __syncthreads();
}

template <int NV, bool VEC, typename T>
DEVINLINE void ld_cols(const T* row, int c, int V, float (&o)[NV]) {
#pragma unroll
  for (int n = 0; n < NV; n += 4) {
    float x[4];
    ld4<T, VEC>(row + c + n, V - c - n, x);
#pragma unroll
    for (int e = 0; e < 4; ++e) o[n + e] = x[e];
  }
}

// grid (chunks, H): U[chunk][h][D][V] = the chunk's own S1, dec[chunk][h][D]
// = e^(sum tot). A unit of work is 16*MD rows by 16*NV columns of U.
template <typename T, int NS, int MD, int NV, bool VEC>
__global__ __launch_bounds__(BLOCK) void gla_chunk_state_kernel(
    const T* __restrict__ proj, GlaSrc p, const int* __restrict__ cu_c,
    float* __restrict__ U, float* __restrict__ dec, int H, int D, int V) {
  constexpr int C = 16 * NS;
  extern __shared__ __align__(16) float lds[];
  __shared__ int far[NS];
  const int ls = row_stride(D);
  float* L = lds;                  // [C][ls]
  float* tot = L + C * ls;         // [NS][ls], later sums over tiles >= a
  float* rs = tot + NS * ls;       // [R][C]
  const int ch = blockIdx.x, h = blockIdx.y;
  const int t0 = cu_c[ch], n = cu_c[ch + 1] - t0;
  chunk_logs<T, NS>(proj, p, t0, n, h, H, D, ls, L, tot, rs, far);
  for (int d = threadIdx.x; d < D; d += BLOCK) {
    float s = 0.f;
#pragma unroll
    for (int a = NS - 1; a >= 0; --a) {
      s += tot[a * ls + d];
      tot[a * ls + d] = s;
    }
    dec[((int64_t)ch * H + h) * D + d] = expf(s);
  }
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int li = lane & 15, quad = lane >> 4;
  const int nd = (D + 16 * MD - 1) / (16 * MD);
  const int nv = (V + 16 * NV - 1) / (16 * NV);
  for (int u = wave; u < nd * nv; u += 4) {
    const int db = (u % nd) * 16 * MD, cb = (u / nd) * 16 * NV;
    const int d0 = db + li * MD, c = cb + li * NV;
    f32x4 acc[MD][NV];
#pragma unroll
    for (int m = 0; m < MD; ++m)
#pragma unroll
      for (int x = 0; x < NV; ++x) acc[m][x] = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < 4 * NS; ++s) {
      const int j = quad * 4 * NS + s;
      float kw[MD], vv[NV];
#pragma unroll
      for (int m = 0; m < MD; ++m) kw[m] = 0.f;
#pragma unroll
      for (int x = 0; x < NV; ++x) vv[x] = 0.f;
      if (j < n) {
        const T* row = proj + (int64_t)(t0 + j) * p.ld;
#pragma unroll
        for (int m = 0; m < MD; ++m)
          if (d0 + m < D)
            kw[m] = ldf<T>(row + p.k_off + h * D + d0 + m) *
                    expf(tot[(j >> 4) * ls + d0 + m] - L[j * ls + d0 + m]);
        ld_cols<NV, VEC, T>(row + p.v_off + h * V, c, V, vv);
      }
#pragma unroll
      for (int m = 0; m < MD; ++m)
#pragma unroll
        for (int x = 0; x < NV; ++x)
          acc[m][x] = __builtin_amdgcn_mfma_f32_16x16x4f32(kw[m], vv[x],
                                                           acc[m][x], 0, 0, 0);
    }
    float* Uc = U + ((int64_t)ch * H + h) * D * V;
#pragma unroll
    for (int m = 0; m < MD; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = db + (quad * 4 + r) * MD + m;
        if (d >= D) continue;
        float* urow = Uc + (int64_t)d * V + c;
#pragma unroll
        for (int x = 0; x < NV; x += 4) {
          if (VEC && c + x + 3 < V) {
            *reinterpret_cast<float4*>(urow + x) =
                make_float4(acc[m][x][r], acc[m][x + 1][r], acc[m][x + 2][r],
                            acc[m][x + 3][r]);
          } else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
              if (c + x + e < V) urow[x + e] = acc[m][x + e][r];
          }
        }
      }
  }
}

// grid (B, H, ceil(D*V / BLOCK)): U holds the chunks' own states on entry
// and the state BEFORE each chunk on exit; the slot receives the state after
// the sequence's last chunk.
__global__ __launch_bounds__(BLOCK) void gla_chain_kernel(
    float* __restrict__ U, const float* __restrict__ dec,
    float* __restrict__ S, const int* __restrict__ chunk_base,
    const int* __restrict__ n_chunks, const int* __restrict__ slots,
    const int* __restrict__ pos0, int H, int D, int V) {
  const int b = blockIdx.x, h = blockIdx.y;
  const int DV = D * V;
  const int e = blockIdx.z * BLOCK + threadIdx.x;
  const int nc = n_chunks[b];
  if (e >= DV || nc <= 0) return;
  const int d = e / V;
  float* Sp = S + ((int64_t)slots[b] * H + h) * DV + e;
  float s = pos0[b] == 0 ? 0.f : *Sp;
  const int c0 = chunk_base[b], c1 = c0 + nc;
  const int64_t su = (int64_t)H * DV, sd = (int64_t)H * D;
  float* up = U + ((int64_t)c0 * H + h) * DV + e;
  const float* dp = dec + ((int64_t)c0 * H + h) * D + d;
  // four chunks' summaries are loaded before they are used
  int c = c0;
  for (; c + 4 <= c1; c += 4) {
    float u[4], a[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      u[i] = up[i * su];
      a[i] = dp[i * sd];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      up[i * su] = s;
      s = a[i] * s + u[i];
    }
    up += 4 * su;
    dp += 4 * sd;
  }
  for (; c < c1; ++c) {
    const float u = *up;
    *up = s;
    s = *dp * s + u;
    up += su;
    dp += sd;
  }
  *Sp = s;
}

// grid (chunks, H): out[t][h][V] from U (the state before each chunk)
template <typename T, int NS, int NV, bool VEC>
__global__ __launch_bounds__(BLOCK) void gla_chunk_out_kernel(
    const T* __restrict__ proj, GlaSrc p, const int* __restrict__ cu_c,
    const float* __restrict__ U, float* __restrict__ out, int H, int D,
    int V) {
  constexpr int C = 16 * NS;
  constexpr int AS = C + 4;        // LDS row stride of A
  extern __shared__ __align__(16) float lds[];
  __shared__ int far[NS];
  const int ls = row_stride(D), dq = quarter(D);
  float* L = lds;                  // [C][ls]
  float* tot = L + C * ls;         // [NS][ls]
  float* A = tot + NS * ls;        // [C][AS]
  float* rs = A + C * AS;          // [R][C]
  const int ch = blockIdx.x, h = blockIdx.y;
  const int t0 = cu_c[ch], n = cu_c[ch + 1] - t0;
  chunk_logs<T, NS>(proj, p, t0, n, h, H, D, ls, L, tot, rs, far);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int li = lane & 15, quad = lane >> 4;
  const T* qh = proj + (int64_t)t0 * p.ld + p.q_off + h * D;
  const T* kh = proj + (int64_t)t0 * p.ld + p.k_off + h * D;

  // ---- A, tile by tile (tiles whose tokens do not exist are skipped)
  for (int u = wave; u < NS * (NS + 1) / 2; u += 4) {
    int a = 0;
    while ((a + 1) * (a + 2) / 2 <= u) ++a;
    const int b = u - a * (a + 1) / 2;
    if (a * 16 >= n) continue;
    f32x4 acc = (f32x4){0.f, 0.f, 0.f, 0.f};
    if (a == b && far[a]) {
      // strong decay inside the tile: every score on its own
      const int j = a * 16 + li;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = a * 16 + quad * 4 + r;
        float s = 0.f;
        if (j <= i && i < n)
          for (int d = 0; d < D; ++d)
            s += ldf<T>(qh + (int64_t)i * p.ld + d) *
                 ldf<T>(kh + (int64_t)j * p.ld + d) *
                 expf(L[i * ls + d] - L[j * ls + d]);
        acc[r] = s * p.qscale;
      }
    } else {
      const int i = a * 16 + li, j = b * 16 + li;
      for (int s = 0; s < dq; s += 4) {
        const int d = quad * dq + s;
        float q[4] = {0.f, 0.f, 0.f, 0.f}, k[4] = {0.f, 0.f, 0.f, 0.f};
        if (i < n) ld4<T, VEC>(qh + (int64_t)i * p.ld + d, D - d, q);
        if (j < n) ld4<T, VEC>(kh + (int64_t)j * p.ld + d, D - d, k);
        const float4 lq = *reinterpret_cast<const float4*>(L + i * ls + d);
        const float4 lk = *reinterpret_cast<const float4*>(L + j * ls + d);
        float eq[4] = {lq.x, lq.y, lq.z, lq.w};
        float ek[4] = {-lk.x, -lk.y, -lk.z, -lk.w};
        if (a != b) {
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            ek[e] += tot[b * ls + d + e];
            for (int m = b + 1; m < a; ++m) eq[e] += tot[m * ls + d + e];
          }
        }
#pragma unroll
        for (int e = 0; e < 4; ++e)
          acc = __builtin_amdgcn_mfma_f32_16x16x4f32(
              q[e] * p.qscale * expf(eq[e]), k[e] * expf(ek[e]), acc, 0, 0, 0);
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = quad * 4 + r;
      A[(a * 16 + i) * AS + b * 16 + li] = (a == b && li > i) ? 0.f : acc[r];
    }
  }
  __syncthreads();

  // ---- outputs: 16 tokens by 16*NV columns per unit
  const int nv = (V + 16 * NV - 1) / (16 * NV);
  const float* Uc = U + ((int64_t)ch * H + h) * D * V;
  for (int u = wave; u < NS * nv; u += 4) {
    const int a = u % NS, c = (u / NS) * 16 * NV + li * NV;
    if (a * 16 >= n) continue;
    f32x4 acc[NV];
#pragma unroll
    for (int x = 0; x < NV; ++x) acc[x] = (f32x4){0.f, 0.f, 0.f, 0.f};
    const int i = a * 16 + li;
    for (int s = 0; s < dq; s += 4) {
      const int d = quad * dq + s;
      float q[4] = {0.f, 0.f, 0.f, 0.f};
      if (i < n) ld4<T, VEC>(qh + (int64_t)i * p.ld + d, D - d, q);
      const float4 lq = *reinterpret_cast<const float4*>(L + i * ls + d);
      float eq[4] = {lq.x, lq.y, lq.z, lq.w};
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        for (int m = 0; m < a; ++m) eq[e] += tot[m * ls + d + e];
        const float qe = q[e] * p.qscale * expf(eq[e]);
        float s0[NV];
#pragma unroll
        for (int x = 0; x < NV; ++x) s0[x] = 0.f;
        if (d + e < D)
          ld_cols<NV, VEC, float>(Uc + (int64_t)(d + e) * V, c, V, s0);
#pragma unroll
        for (int x = 0; x < NV; ++x)
          acc[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(qe, s0[x], acc[x], 0,
                                                        0, 0);
      }
    }
    for (int b = 0; b <= a; ++b) {
      const float4 a4 =
          *reinterpret_cast<const float4*>(A + i * AS + b * 16 + quad * 4);
      const float av[4] = {a4.x, a4.y, a4.z, a4.w};
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int j = b * 16 + quad * 4 + e;
        float vv[NV];
#pragma unroll
        for (int x = 0; x < NV; ++x) vv[x] = 0.f;
        if (j < n)
          ld_cols<NV, VEC, T>(
              proj + (int64_t)(t0 + j) * p.ld + p.v_off + h * V, c, V, vv);
#pragma unroll
        for (int x = 0; x < NV; ++x)
          acc[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(av[e], vv[x], acc[x],
                                                        0, 0, 0);
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = a * 16 + quad * 4 + r;
      if (t >= n) continue;
      float* orow = out + ((int64_t)(t0 + t) * H + h) * V + c;
#pragma unroll
      for (int x = 0; x < NV; x += 4) {
        if (VEC && c + x + 3 < V) {
          *reinterpret_cast<float4*>(orow + x) = make_float4(
              acc[x][r], acc[x + 1][r], acc[x + 2][r], acc[x + 3][r]);
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (c + x + e < V) orow[x + e] = acc[x + e][r];
        }
      }
    }
  }
}

size_t scan_smem(int DP, int R) {
  return sizeof(float) *
         ((size_t)RT * (3 * DP + VT + 4 * VT) + (size_t)RT * R);
}

size_t chunk_smem(int NS, int D, int R, bool with_a) {
  const size_t C = 16 * NS, ls = row_stride(D);
  return sizeof(float) *
         (C * ls + NS * ls + C * R + (with_a ? C * (C + 4) : 0));
}

constexpr size_t LDS_MAX = 64 * 1024 - 64;

template <typename T, int NS, int NV, bool VEC>
void launch_chunks(const T* proj, const GlaSrc& p, const int* cu_c, int NC,
                   const int* base, const int* cnt, const int* slots,
                   const int* pos0, int B, float* S, float* U, float* dec,
                   float* out, int H, int D, int V, hipStream_t stream) {
  dim3 grid(NC, H), block(BLOCK);
  const size_t sm = chunk_smem(NS, D, p.R, false);
#define TL_GLA_ST(MD)                                                        \
  hipLaunchKernelGGL((gla_chunk_state_kernel<T, NS, MD, NV, VEC>), grid,     \
                     block, sm, stream, proj, p, cu_c, U, dec, H, D, V)
  if (D <= 64) TL_GLA_ST(1);
  else if (D <= 128) TL_GLA_ST(2);
  else TL_GLA_ST(4);
#undef TL_GLA_ST
  hipLaunchKernelGGL(gla_chain_kernel,
                     dim3(B, H, (D * V + BLOCK - 1) / BLOCK), block, 0, stream,
                     U, (const float*)dec, S, base, cnt, slots, pos0, H, D, V);
  hipLaunchKernelGGL((gla_chunk_out_kernel<T, NS, NV, VEC>), grid, block,
                     chunk_smem(NS, D, p.R, true), stream, proj, p, cu_c,
                     (const float*)U, out, H, D, V);
}

template <typename T>
int chunks_any(const T* proj, const GlaSrc& p, const int* cu_c, int NC,
               const int* base, const int* cnt, const int* slots,
               const int* pos0, int B, float* S, float* U, float* dec,
               float* out, int H, int D, int V, int C, hipStream_t stream) {
  const bool vec = D % 4 == 0 && V % 4 == 0 && p.ld % 4 == 0 &&
                   p.q_off % 4 == 0 && p.k_off % 4 == 0 && p.v_off % 4 == 0;
#define TL_GLA_C(NS, NV, VEC)                                                \
  launch_chunks<T, NS, NV, VEC>(proj, p, cu_c, NC, base, cnt, slots, pos0, B, \
                                S, U, dec, out, H, D, V, stream)
#define TL_GLA_CV(NS, NV)              \
  if (vec) TL_GLA_C(NS, NV, true);     \
  else TL_GLA_C(NS, NV, false)
  if (C == 64) {
    if (V <= 64) { TL_GLA_CV(4, 4); }
    else { TL_GLA_CV(4, 8); }
  } else {
    if (V <= 64) { TL_GLA_CV(2, 4); }
    else { TL_GLA_CV(2, 8); }
  }
#undef TL_GLA_CV
#undef TL_GLA_C
  return 0;
}

}  // namespace

extern "C" {

// 1 if tl_gla_chunks serves the shape with chunks of C tokens
int tl_gla_chunks_ok(int D, int R, int C) {
  if (C != 64 && C != 32) return 0;
  if (D < 1 || D > 256 || R < 1) return 0;
  return chunk_smem(C / 16, D, R, true) <= LDS_MAX ? 1 : 0;
}

// returns 0 on success, 1 if the shape is outside what the kernels serve
int tl_gla_chunks(const void* proj, int ld, int q_off, int k_off, int v_off,
                  int r_off, const void* a2t, const void* bias, int R,
                  float inv_tau, float qscale, void* S, const void* cu_c,
                  int NC, const void* base, const void* cnt, const void* slots,
                  const void* pos0, int B, void* U, void* dec, void* out,
                  int H, int D, int V, int C, int is_f32,
                  hipStream_t stream) {
  if (!tl_gla_chunks_ok(D, R, C) || H <= 0 || V <= 0) return 1;
  if (NC <= 0 || B <= 0) return 0;
  GlaSrc p{ld, q_off, k_off, v_off, r_off, (const float*)a2t,
           (const float*)bias, R, inv_tau, qscale};
  if (is_f32)
    return chunks_any<float>((const float*)proj, p, (const int*)cu_c, NC,
                             (const int*)base, (const int*)cnt,
                             (const int*)slots, (const int*)pos0, B,
                             (float*)S, (float*)U, (float*)dec, (float*)out,
                             H, D, V, C, stream);
  return chunks_any<bf16>((const bf16*)proj, p, (const int*)cu_c, NC,
                          (const int*)base, (const int*)cnt,
                          (const int*)slots, (const int*)pos0, B, (float*)S,
                          (float*)U, (float*)dec, (float*)out, H, D, V, C,
                          stream);
}

// returns 0 on success, 1 if the launch cannot be made
int tl_gla_scan(const void* proj, int ld, int q_off, int k_off, int v_off,
                int r_off, const void* a2t, const void* bias, int R,
                float inv_tau, float qscale, void* S, const void* cu,
                const void* slots, const void* pos0, void* out, int B, int H,
                int D, int V, int is_f32, hipStream_t stream) {
  if (B <= 0 || H <= 0 || D <= 0 || V <= 0 || R <= 0) return 1;
  GlaSrc p{ld, q_off, k_off, v_off, r_off, (const float*)a2t,
           (const float*)bias, R, inv_tau, qscale};
  dim3 grid(B, H, (V + VT - 1) / VT), block(BLOCK);
#define TL_GS(TT, DR)                                                        \
  hipLaunchKernelGGL((gla_scan_kernel<TT, DR>), grid, block,                 \
                     scan_smem(4 * DR, R), stream, (const TT*)proj, p,       \
                     (float*)S, (const int*)cu, (const int*)slots,           \
                     (const int*)pos0, (float*)out, H, D, V)
#define TL_GS_T(DR)                                \
  if (D <= 4 * DR && scan_smem(4 * DR, R) <= LDS_MAX) { \
    if (is_f32) TL_GS(float, DR);                  \
    else TL_GS(bf16, DR);                          \
    return 0;                                      \
  }
  TL_GS_T(8)
  TL_GS_T(16)
  TL_GS_T(32)
  TL_GS_T(64)
#undef TL_GS_T
#undef TL_GS
  const size_t gsmem = sizeof(float) * 3 * (size_t)D;
  if (gsmem > LDS_MAX) return 1;
  dim3 g2(B, H);
  if (is_f32)
    hipLaunchKernelGGL(gla_scan_generic_kernel<float>, g2, block, gsmem,
                       stream, (const float*)proj, p, (float*)S,
                       (const int*)cu, (const int*)slots, (const int*)pos0,
                       (float*)out, H, D, V);
  else
    hipLaunchKernelGGL(gla_scan_generic_kernel<bf16>, g2, block, gsmem,
                       stream, (const bf16*)proj, p, (float*)S,
                       (const int*)cu, (const int*)slots, (const int*)pos0,
                       (float*)out, H, D, V);
  return 0;
}

}  // extern "C"
