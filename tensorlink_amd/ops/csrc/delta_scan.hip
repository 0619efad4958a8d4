// Gated delta rule (one decay per key channel and token) over ragged
// sequences (gfx950).
//
// Per head (q, k unit vectors, q also times D^-1/2):
//     log g_t = -exp(A_log) softplus(r_t A2 + dt_bias)            [D], <= 0
//     S  <- diag(g_t) S_(t-1)                    (S is [D, V], fp32, per slot)
//     u_t = beta_t (v_t - S^T k_t);  S_t = S + k_t u_t^T;  o_t = S_t^T q_t
// q, k, v are columns of the convolved projection (fp32; q and k of head h
// are those of group h / (H / G)), r the low-rank columns of the raw
// projection (bf16 or fp32), beta = sigmoid of an fp32 column. Unit norms,
// decays and everything behind them are fp32 and never written to memory
// outside the chunk form's scratch.
//
// tl_delta_scan walks the tokens in order (decoding, short portions). One
// block per (sequence, head, 64 value columns), columns of S are
// independent. A wave owns 16 columns: lane (c, g) holds column c of S for DR
// consecutive rows from g * DR, so the two dot products of a token (with k
// before the write, with q after it) are closed by two lane exchanges each
// and the token loop has no barrier. Key sizes beyond the register budget
// take the generic kernel (state in the slot's memory).
//
// Long prompt portions take the chunk form: chunks of C = 32 tokens in two
// tiles of 16. With L_t the running sum of log g inside the chunk,
//     A_ts = beta_t sum_d k_td k_sd e^(L_td - L_sd)               (s < t)
//     (I + A) U = diag(beta) V - diag(beta) [K e^L] S0
//     O  = [Q e^L] S0 + B U,  B_ts = sum_d q_td k_sd e^(L_td - L_sd)  (s <= t)
//     S1 = e^(L_C) S0 + [K e^(L_C - L)]^T U
// tl_delta_chunk_prep computes, per chunk and head, W = (I + A)^-1 diag(beta)
// [K e^L] and U0 = (I + A)^-1 diag(beta) V by block forward substitution (the
// 16 x 16 diagonal blocks are inverted), B, [Q e^L], [K e^(L_C - L)]^T and
// e^(L_C). tl_delta_chunk_chain then walks a sequence's chunks with
// U = U0 - W S0; one block per (sequence, head, 16 value columns).
// Exponents: with l the running sum inside a token's own tile and tot_a a
// tile's total, products between tiles use e^(l_i + sum of tiles between) and
// e^(tot_b - l_j), all exponents <= 0. Inside a tile the product factors as
// e^(l_i) e^(-l_j) while the tile's decay stays within LOG_RANGE; otherwise
// it is summed with e^(l_i - l_j) directly. All products run on the fp32
// MFMA (16x16x4).
//
// MFMA operands: lane (i = lane & 15, g = lane >> 4) supplies A[i][k] and
// B[k][i] of one k per instruction, and receives rows 4g .. 4g + 3 of column
// i. The order of the k's is free: group g takes k = 4g + s at step s, so an
// accumulator is the B operand of the next product as it stands.

#include "common.hpp"

namespace {

constexpr int BLOCK = 256;
constexpr int RT = 8;               // tokens per round of the scan
constexpr int VT = 64;              // value columns per block of the scan
constexpr int CHUNK = 32;           // tokens per chunk
constexpr int CT = 16;              // value columns per block of the chain
constexpr int CS = CT + 4;          // their LDS row stride
constexpr float LOG_RANGE = 60.f;   // e^60 * e^60 is inside fp32
// chunk form: a token's log decay is cut here. e^-60 of a memory is nothing
// beside what any token writes, and the running sums, whose differences are
// taken, keep their digits.
constexpr float LOG_FLOOR = -60.f;

using f32x4 = __attribute__((ext_vector_type(4))) float;

template <typename T> DEVINLINE float ldf(const T* p);
template <> DEVINLINE float ldf<float>(const float* p) { return *p; }
template <> DEVINLINE float ldf<bf16>(const bf16* p) { return bf2f(*p); }

DEVINLINE float softplus_f(float z) {
  return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z)));
}

struct DeltaSrc {
  const float* x;      // [T, ldx] convolved q | k | v
  int ldx, q_off, k_off, v_off;
  int ldr, r_off, R;   // low-rank decay columns of the raw projection
  const float* b;      // [T, ldb] raw beta
  int ldb, b_off;
  const float* a2t;    // [R][H*D]
  const float* dt_bias;  // [H*D]
  const float* A_log;  // [H]
  float qscale;
  int rep;             // heads per q/k group
};

// ------------------------------------------------------------------ scan
template <typename T, int DR>
__global__ __launch_bounds__(BLOCK) void delta_scan_kernel(
    const T* __restrict__ proj, DeltaSrc p, float* __restrict__ S,
    const int* __restrict__ cu, const int* __restrict__ slots,
    const int* __restrict__ pos0, float* __restrict__ out, int H, int D,
    int V) {
  constexpr int GS = DR + 4;        // LDS stride of one lane group's rows
  constexpr int DP = 4 * GS;
  extern __shared__ __align__(16) float lds[];
  // lds: qs | ks | gs [RT][DP] | vs[RT][VT] | bs[RT] | rs[RT][R]
  float* qs = lds;
  float* ks = qs + RT * DP;
  float* gs = ks + RT * DP;
  float* vs = gs + RT * DP;
  float* bs = vs + RT * VT;
  float* rs = bs + RT;
  const int b = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * VT;
  const int t0 = cu[b], t1 = cu[b + 1];
  if (t1 <= t0) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int g = lane >> 4, cl = wave * 16 + (lane & 15);
  const int c = c0 + cl;
  const int hq = h / p.rep;
  float* Sh = S + ((int64_t)slots[b] * H + h) * D * V;
  const bool fresh = pos0[b] == 0;
  const float ea = -expf(p.A_log[h]);
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
      rs[i] = ldf<T>(proj + (int64_t)(tb + tt) * p.ldr + p.r_off + r);
    }
    for (int i = threadIdx.x; i < nt * VT; i += BLOCK) {
      const int tt = i / VT, e = i & (VT - 1);
      vs[i] = c0 + e < V
                  ? p.x[(int64_t)(tb + tt) * p.ldx + p.v_off + h * V + c0 + e]
                  : 0.f;
    }
    if (threadIdx.x < nt)
      bs[threadIdx.x] =
          1.f / (1.f + expf(-p.b[(int64_t)(tb + threadIdx.x) * p.ldb +
                                 p.b_off + h]));
    __syncthreads();
    // decays: four lanes per channel, eight loads in flight each
    for (int i = threadIdx.x; i < nt * 4 * DR * 4; i += BLOCK) {
      const int j = i & 3, w = i >> 2;
      const int tt = w / (4 * DR), d = w - tt * (4 * DR);
      const int hd = h * D + min(d, D - 1);
      float z = 0.f;
      for (int r0 = j; r0 < p.R; r0 += 32) {
        float x[8];
#pragma unroll
        for (int e = 0; e < 8; ++e)
          x[e] = p.a2t[(int64_t)min(r0 + 4 * e, p.R - 1) * H * D + hd];
#pragma unroll
        for (int e = 0; e < 8; ++e)
          if (r0 + 4 * e < p.R) z += rs[tt * p.R + r0 + 4 * e] * x[e];
      }
      z += __shfl_xor(z, 1, WAVE_SIZE);
      z += __shfl_xor(z, 2, WAVE_SIZE);
      if (j == 0)
        gs[tt * DP + (d / DR) * GS + d % DR] =
            d < D ? expf(ea * softplus_f(z + p.dt_bias[hd])) : 1.f;
    }
    // unit vectors, one wave per token
    for (int tt = wave; tt < nt; tt += BLOCK / WAVE_SIZE) {
      const float* row = p.x + (int64_t)(tb + tt) * p.ldx;
      constexpr int NP = (4 * DR + 63) / 64;
      float qv[NP], kv[NP], sq = 0.f, sk = 0.f;
#pragma unroll
      for (int i = 0; i < NP; ++i) {
        const int d = i * 64 + lane;
        qv[i] = d < D ? row[p.q_off + hq * D + d] : 0.f;
        kv[i] = d < D ? row[p.k_off + hq * D + d] : 0.f;
        sq += qv[i] * qv[i];
        sk += kv[i] * kv[i];
      }
      const float rq = p.qscale / sqrtf(wave_reduce_sum(sq) + 1e-6f);
      const float rk = 1.f / sqrtf(wave_reduce_sum(sk) + 1e-6f);
#pragma unroll
      for (int i = 0; i < NP; ++i) {
        const int d = i * 64 + lane;
        if (d < 4 * DR) {
          const int o = tt * DP + (d / DR) * GS + d % DR;
          qs[o] = qv[i] * rq;
          ks[o] = kv[i] * rk;
        }
      }
    }
    __syncthreads();
    for (int tt = 0; tt < nt; ++tt) {
      const float4* g4 =
          reinterpret_cast<const float4*>(gs + tt * DP + g * GS);
      const float4* k4 =
          reinterpret_cast<const float4*>(ks + tt * DP + g * GS);
      const float4* q4 =
          reinterpret_cast<const float4*>(qs + tt * DP + g * GS);
      float read = 0.f;
#pragma unroll
      for (int r = 0; r < DR / 4; ++r) {
        const float4 a = g4[r], k = k4[r];
        st[4 * r + 0] *= a.x;
        st[4 * r + 1] *= a.y;
        st[4 * r + 2] *= a.z;
        st[4 * r + 3] *= a.w;
        read += st[4 * r + 0] * k.x + st[4 * r + 1] * k.y +
                st[4 * r + 2] * k.z + st[4 * r + 3] * k.w;
      }
      read += __shfl_xor(read, 16, WAVE_SIZE);
      read += __shfl_xor(read, 32, WAVE_SIZE);
      const float u = bs[tt] * (vs[tt * VT + cl] - read);
      float acc = 0.f;
#pragma unroll
      for (int r = 0; r < DR / 4; ++r) {
        const float4 k = k4[r], q = q4[r];
        st[4 * r + 0] += k.x * u;
        st[4 * r + 1] += k.y * u;
        st[4 * r + 2] += k.z * u;
        st[4 * r + 3] += k.w * u;
        acc += st[4 * r + 0] * q.x + st[4 * r + 1] * q.y +
               st[4 * r + 2] * q.z + st[4 * r + 3] * q.w;
      }
      acc += __shfl_xor(acc, 16, WAVE_SIZE);
      acc += __shfl_xor(acc, 32, WAVE_SIZE);
      if (g == 0 && c < V) out[((int64_t)(tb + tt) * H + h) * V + c] = acc;
    }
  }
#pragma unroll
  for (int r = 0; r < DR; ++r) {
    const int d = g * DR + r;
    if (d < D && c < V) Sh[(int64_t)d * V + c] = st[r];
  }
}

// Any key size: the state stays in the slot's memory; thread c owns the
// columns c, c + BLOCK, ... and walks all rows twice for every token.
template <typename T>
__global__ __launch_bounds__(BLOCK) void delta_scan_generic_kernel(
    const T* __restrict__ proj, DeltaSrc p, float* __restrict__ S,
    const int* __restrict__ cu, const int* __restrict__ slots,
    const int* __restrict__ pos0, float* __restrict__ out, int H, int D,
    int V) {
  extern __shared__ __align__(16) float lds[];  // gs[D] | ks[D] | qs[D]
  __shared__ float red[BLOCK / WAVE_SIZE], red2[BLOCK / WAVE_SIZE];
  float* gs = lds;
  float* ks = gs + D;
  float* qs = ks + D;
  const int b = blockIdx.x, h = blockIdx.y;
  const int t0 = cu[b], t1 = cu[b + 1];
  if (t1 <= t0) return;
  const int hq = h / p.rep;
  const float ea = -expf(p.A_log[h]);
  float* Sh = S + ((int64_t)slots[b] * H + h) * D * V;
  if (pos0[b] == 0)
    for (int c = threadIdx.x; c < V; c += BLOCK)
      for (int d = 0; d < D; ++d) Sh[(int64_t)d * V + c] = 0.f;
  for (int t = t0; t < t1; ++t) {
    __syncthreads();
    const float* row = p.x + (int64_t)t * p.ldx;
    float sq = 0.f, sk = 0.f;
    for (int d = threadIdx.x; d < D; d += BLOCK) {
      const int hd = h * D + d;
      const float q = row[p.q_off + hq * D + d];
      const float k = row[p.k_off + hq * D + d];
      sq += q * q;
      sk += k * k;
      qs[d] = q;
      ks[d] = k;
      float z = p.dt_bias[hd];
      for (int r = 0; r < p.R; ++r)
        z += ldf<T>(proj + (int64_t)t * p.ldr + p.r_off + r) *
             p.a2t[(int64_t)r * H * D + hd];
      gs[d] = expf(ea * softplus_f(z));
    }
    const float tq = block_reduce_sum<BLOCK / WAVE_SIZE>(sq, red);
    const float tk = block_reduce_sum<BLOCK / WAVE_SIZE>(sk, red2);
    const float rq = p.qscale / sqrtf(tq + 1e-6f);
    const float rk = 1.f / sqrtf(tk + 1e-6f);
    const float beta =
        1.f / (1.f + expf(-p.b[(int64_t)t * p.ldb + p.b_off + h]));
    for (int c = threadIdx.x; c < V; c += BLOCK) {
      float read = 0.f;
      for (int d = 0; d < D; ++d)
        read += gs[d] * Sh[(int64_t)d * V + c] * (ks[d] * rk);
      const float u = beta * (row[p.v_off + h * V + c] - read);
      float acc = 0.f;
      for (int d = 0; d < D; ++d) {
        const float s = gs[d] * Sh[(int64_t)d * V + c] + ks[d] * rk * u;
        Sh[(int64_t)d * V + c] = s;
        acc += s * (qs[d] * rq);
      }
      out[((int64_t)t * H + h) * V + c] = acc;
    }
  }
}

// ----------------------------------------------------------- chunk form
// The caller's scratch, all fp32, per (chunk, head); DP = 16 * DT >= D,
// VP = V rounded up to CT:
struct DeltaScratch {
  float* W;     // [C][DP]
  float* Q;     // [C][DP]   q e^L
  float* Kt;    // [DP][C]   (k e^(L_C - L)) transposed
  float* B;     // [C][C]    lower triangle with diagonal
  float* U;     // [C][VP]
  float* dec;   // [DP]      e^(L_C)
};
// The matrices are cut into 16 x 16 tiles, row tiles first, and a tile is
// stored in the order the chain's waves hold it, four elements per lane, so
// that every load is one contiguous KiB: W, Q, Kt and B as A operands (lane
// (i, g) has row i, columns 4g .. 4g + 3), U as an accumulator (rows 4g ..
// 4g + 3 of column i).
DEVINLINE int operand_at(int row, int col) {     // inside a tile
  return ((col >> 2) * 16 + row) * 4 + (col & 3);
}

// A barrier for exchanges through LDS only: global loads stay in flight.
DEVINLINE void lds_barrier() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "workgroup", "local");
  __builtin_amdgcn_s_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup", "local");
}

DEVINLINE f32x4 mfma4(const float4& a, float b0, float b1, float b2, float b3,
                      f32x4 c) {
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b0, c, 0, 0, 0);
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b1, c, 0, 0, 0);
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b2, c, 0, 0, 0);
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b3, c, 0, 0, 0);
}

// grid (chunks, H). LDS arrays of rows [token][channel]: first the raw q and
// k and the running logs, then, in place, q e^l, k e^l and k e^(tot - l)
template <typename T, int NS, int DT>
__global__ __launch_bounds__(BLOCK, 4) void delta_chunk_prep_kernel(
    const T* __restrict__ proj, DeltaSrc p, const int* __restrict__ cu_c,
    DeltaScratch s, int H, int D, int V, int VP) {
  static_assert(NS == 2, "no tile lies between two others");
  constexpr int C = 16 * NS, DP = 16 * DT;
  constexpr int LS = DP + 4, AS = C + 4;
  extern __shared__ __align__(16) float lds[];
  __shared__ int far[NS];
  __shared__ float qn[C], kn[C], bt[C];
  float* Qe = lds;                 // [C][LS]
  float* Ke = Qe + C * LS;
  float* Kd = Ke + C * LS;         // first L, the running logs inside a tile
  float* tot = Kd + C * LS;        // [NS][LS] a tile's sum of logs
  float* Et = tot + NS * LS;       // [NS][LS] e^tot
  float* Ei = Et + NS * LS;        // [NS][LS] e^(-tot) (tiles in range only)
  float* A = Ei + NS * LS;        // [C][AS]; first the low-rank rows [C][RS]
  const int ch = blockIdx.x, h = blockIdx.y, hq = h / p.rep;
  const int t0 = cu_c[ch], n = cu_c[ch + 1] - t0;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int li = lane & 15, quad = lane >> 4;
  const float* qh = p.x + (int64_t)t0 * p.ldx + p.q_off + hq * D;
  const float* kh = p.x + (int64_t)t0 * p.ldx + p.k_off + hq * D;
  const float* vh = p.x + (int64_t)t0 * p.ldx + p.v_off + h * V;
  const int64_t ci = (int64_t)ch * H + h;

  // ---- stage: low-rank rows, raw q and k, step sizes
  if (threadIdx.x < NS) far[threadIdx.x] = 0;
  const int RP = (p.R + 15) / 16 * 16, RS = RP + 4;
  // (loads are unconditional, from the nearest place that exists, and what
  // does not exist is cleared afterwards: no branch around a load, so that
  // all of them are in flight together)
  {
    constexpr int TPT = BLOCK / C;   // threads per token
    const int t = threadIdx.x / TPT, j = threadIdx.x % TPT;
    const T* row = proj + (int64_t)(t0 + min(t, n - 1)) * p.ldr + p.r_off;
    for (int r0 = 0; r0 < RP; r0 += TPT * 8) {
      float x[8];
#pragma unroll
      for (int e = 0; e < 8; ++e)
        x[e] = ldf<T>(row + min(r0 + e * TPT + j, p.R - 1));
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int r = r0 + e * TPT + j;
        if (r < RP) A[t * RS + r] = t < n && r < p.R ? x[e] : 0.f;
      }
    }
  }
  {
    constexpr int IT = C * DP / BLOCK;
    float q[IT], k[IT];
#pragma unroll
    for (int i = 0; i < IT; ++i) {
      const int e = i * BLOCK + threadIdx.x, t = e / DP, d = e - t * DP;
      const int64_t o = (int64_t)min(t, n - 1) * p.ldx + min(d, D - 1);
      q[i] = qh[o];
      k[i] = kh[o];
    }
#pragma unroll
    for (int i = 0; i < IT; ++i) {
      const int e = i * BLOCK + threadIdx.x, t = e / DP, d = e - t * DP;
      const bool in = t < n && d < D;
      Qe[t * LS + d] = in ? q[i] : 0.f;
      Ke[t * LS + d] = in ? k[i] : 0.f;
    }
  }
  if (threadIdx.x < C)
    bt[threadIdx.x] =
        threadIdx.x < n
            ? 1.f / (1.f + expf(-p.b[(int64_t)(t0 + threadIdx.x) * p.ldb +
                                     p.b_off + h]))
            : 0.f;
  __syncthreads();
  // ---- norms (four tokens per wave and step) and decays
  for (int t = wave * 4 + quad; t < C; t += 16) {
    float sq = 0.f, sk = 0.f;
#pragma unroll
    for (int d = 0; d < DP; d += 16) {
      const float q = Qe[t * LS + d + li], k = Ke[t * LS + d + li];
      sq += q * q;
      sk += k * k;
    }
#pragma unroll
    for (int off = 8; off > 0; off >>= 1) {
      sq += __shfl_xor(sq, off, WAVE_SIZE);
      sk += __shfl_xor(sk, off, WAVE_SIZE);
    }
    if (li == 0) {
      qn[t] = p.qscale / sqrtf(sq + 1e-6f);
      kn[t] = 1.f / sqrtf(sk + 1e-6f);
    }
  }
  const float ea = -expf(p.A_log[h]);
  for (int u = wave; u < NS * DT; u += 4) {
    const int a = u / DT, d = (u - a * DT) * 16 + li;
    const bool in = d < D;
    f32x4 z = (f32x4){0.f, 0.f, 0.f, 0.f};
    const float* rr = A + (a * 16 + li) * RS + quad * 4;
    // rows beyond R meet zeros of the other operand, channels beyond D are
    // never used
    const float* w2 = p.a2t + h * D + min(d, D - 1);
    const float bz = p.dt_bias[h * D + min(d, D - 1)];
    for (int r0 = 0; r0 < RP; r0 += 64) {
      float w[16];
#pragma unroll
      for (int e = 0; e < 16; ++e) {
        const int r = r0 + (e >> 2) * 16 + quad * 4 + (e & 3);
        w[e] = w2[(int64_t)min(r, p.R - 1) * H * D];
      }
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (r0 + e * 16 < RP) {
          const float4 x = *reinterpret_cast<const float4*>(rr + r0 + e * 16);
          z = mfma4(x, w[4 * e], w[4 * e + 1], w[4 * e + 2], w[4 * e + 3], z);
        }
    }
    // running sums over the tile's 16 tokens: four in this lane, then the
    // lanes of the same channel
    float run[4], sum = 0.f;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      if (in && a * 16 + quad * 4 + r < n)
        sum += fmaxf(ea * softplus_f(z[r] + bz), LOG_FLOOR);
      run[r] = sum;
    }
    float o = __shfl_up(sum, 16, WAVE_SIZE);
    if (quad >= 1) sum += o;
    o = __shfl_up(sum, 32, WAVE_SIZE);
    if (quad >= 2) sum += o;
    o = __shfl_up(sum, 16, WAVE_SIZE);
    const float before = quad >= 1 ? o : 0.f;
#pragma unroll
    for (int r = 0; r < 4; ++r)
      Kd[(a * 16 + quad * 4 + r) * LS + d] = before + run[r];
    if (quad == 3) {
      tot[a * LS + d] = sum;
      Et[a * LS + d] = expf(sum);
      Ei[a * LS + d] = expf(-sum);
      if (sum < -LOG_RANGE) far[a] = 1;    // same value from every writer
    }
  }
  __syncthreads();

  // ---- scores: A (strictly lower, times beta) into LDS, B to memory
  float* Bc = s.B + ci * C * C;
  auto put = [&](int a, int b, const f32x4& ak, const f32x4& aq) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = a * 16 + quad * 4 + r, j = b * 16 + li;
      A[i * AS + j] = j < i ? ak[r] * bt[i] : 0.f;
      Bc[(a * NS + b) * 256 + operand_at(quad * 4 + r, li)] =
          j <= i ? aq[r] : 0.f;
    }
  };
  // diagonal tiles of strong decay: every score on its own, while the raw
  // vectors and the logs are here
  if (wave < NS && far[wave]) {
    const int a = wave, j = a * 16 + li;
    f32x4 ak, aq;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = a * 16 + quad * 4 + r;
      float sk = 0.f, sq = 0.f;
      if (j <= i)
        for (int d = 0; d < D; ++d) {
          const float w =
              Ke[j * LS + d] * expf(Kd[i * LS + d] - Kd[j * LS + d]);
          sk += Ke[i * LS + d] * w;
          sq += Qe[i * LS + d] * w;
        }
      ak[r] = sk * kn[j] * kn[i];
      aq[r] = sq * kn[j] * qn[i];
    }
    put(a, a, ak, aq);
  }
  __syncthreads();
  for (int i = threadIdx.x; i < C * DP; i += BLOCK) {
    const int t = i / DP, o = t * LS + (i - t * DP);
    const int tt = (t >> 4) * LS + (i - t * DP);
    const float l = Kd[o], k = Ke[o] * kn[t];
    const float el = __expf(l), ed = __expf(tot[tt] - l);
    Qe[o] *= qn[t] * el;
    Ke[o] = k * el;
    Kd[o] = k * ed;
  }
  __syncthreads();
  for (int u = wave; u < NS * NS; u += 4) {
    const int a = u / NS, b = u - a * NS;
    if (a == b && far[a]) continue;
    f32x4 ak = (f32x4){0.f, 0.f, 0.f, 0.f}, aq = ak;
    if (b <= a && a * 16 < n) {
      const float* qi = Qe + (a * 16 + li) * LS + quad * 4;
      const float* ki = Ke + (a * 16 + li) * LS + quad * 4;
      const float* kj = Kd + (b * 16 + li) * LS + quad * 4;
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) {
        const float4 q = *reinterpret_cast<const float4*>(qi + dt * 16);
        const float4 k = *reinterpret_cast<const float4*>(ki + dt * 16);
        float4 y = *reinterpret_cast<const float4*>(kj + dt * 16);
        if (a == b) {                // inside a tile e^(-l) alone
          const float4 e = *reinterpret_cast<const float4*>(
              Ei + a * LS + dt * 16 + quad * 4);
          y.x *= e.x;
          y.y *= e.y;
          y.z *= e.z;
          y.w *= e.w;
        }
        ak = mfma4(k, y.x, y.y, y.z, y.w, ak);
        aq = mfma4(q, y.x, y.y, y.z, y.w, aq);
      }
    }
    put(a, b, ak, aq);
  }
  __syncthreads();

  // ---- inverses of the diagonal blocks I + A_aa, in place: lane j < 16
  // solves column j by forward substitution
  if (wave < NS) {
    float* Aa = A + (wave * 16) * AS + wave * 16;
    float x[16];
    // every lane computes; lanes beyond 15 repeat the first ones
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float v = i == li ? 1.f : 0.f;
#pragma unroll
      for (int m = 0; m < i; ++m) v -= Aa[i * AS + m] * x[m];
      x[i] = v;
    }
    __builtin_amdgcn_wave_barrier();
    if (lane < 16)
#pragma unroll
      for (int i = 0; i < 16; ++i) Aa[i * AS + li] = x[i];
  }
  __syncthreads();

  // ---- W and U0: strips of 16 columns, block forward substitution
  float* Wc = s.W + ci * C * DP;
  float* Uc = s.U + ci * C * VP;
  for (int u = wave; u < DT + VP / 16; u += 4) {
    const bool isw = u < DT;
    const int col = (isw ? u : u - DT) * 16 + li;
    float v0[NS][4];
    if (!isw) {
#pragma unroll
      for (int a = 0; a < NS; ++a)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          v0[a][r] = vh[(int64_t)min(a * 16 + quad * 4 + r, n - 1) * p.ldx +
                        min(col, V - 1)];
    }
    f32x4 X[NS];
#pragma unroll
    for (int a = 0; a < NS; ++a) {
      f32x4 y;
      const float eb = isw && a ? Et[col] : 1.f;     // the tile before
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = a * 16 + quad * 4 + r;
        float v = 0.f;
        if (isw) v = Ke[i * LS + col] * eb;
        else v = col < V ? v0[a][r] : 0.f;
        y[r] = v * bt[i];            // 0 beyond the chunk's tokens
      }
#pragma unroll
      for (int b = 0; b < a; ++b) {
        const float4 f = *reinterpret_cast<const float4*>(
            A + (a * 16 + li) * AS + b * 16 + quad * 4);
        y = mfma4(f, -X[b][0], -X[b][1], -X[b][2], -X[b][3], y);
      }
      const float4 f = *reinterpret_cast<const float4*>(
          A + (a * 16 + li) * AS + a * 16 + quad * 4);
      const f32x4 z = mfma4(f, y[0], y[1], y[2], y[3],
                            (f32x4){0.f, 0.f, 0.f, 0.f});
      X[a] = z;
      if (isw) {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          Wc[(a * DT + u) * 256 + operand_at(quad * 4 + r, li)] = z[r];
      } else {
        *reinterpret_cast<float4*>(
            Uc + ((a * (VP / 16) + u - DT) * 64 + lane) * 4) =
            make_float4(z[0], z[1], z[2], z[3]);
      }
    }
  }

  // ---- q e^L, (k e^(L_C - L))^T and e^(L_C)
  float* Qc = s.Q + ci * C * DP;
#pragma unroll
  for (int u = wave; u < NS * DT; u += 4) {
    const int a = u / DT, d = (u - a * DT) * 16 + quad * 4;
    float4 x = *reinterpret_cast<const float4*>(Qe + (a * 16 + li) * LS + d);
    if (a) {
      const float4 e = *reinterpret_cast<const float4*>(Et + d);
      x.x *= e.x;
      x.y *= e.y;
      x.z *= e.z;
      x.w *= e.w;
    }
    *reinterpret_cast<float4*>(Qc + (u * 64 + lane) * 4) = x;
  }
  float* Kc = s.Kt + ci * C * DP;
#pragma unroll
  for (int u = wave; u < NS * DT; u += 4) {
    const int dt = u / NS, a = u - dt * NS, d = dt * 16 + li;
    const float e = a == 0 ? Et[LS + d] : 1.f;
    const float* kp = Kd + (a * 16 + quad * 4) * LS + d;
    *reinterpret_cast<float4*>(Kc + (u * 64 + lane) * 4) = make_float4(
        kp[0] * e, kp[LS] * e, kp[2 * LS] * e, kp[3 * LS] * e);
  }
  for (int d = threadIdx.x; d < DP; d += BLOCK)
    s.dec[ci * DP + d] = Et[d] * Et[LS + d];
}

// what one wave reads of a chunk's scratch
template <int NS, int DT, int NK>
struct ChainFrag {
  float4 wq[DT];                     // its token tile's rows of W or Q
  float4 u0;
  float4 b[NS];
  float4 kt[NK][NS], dec[NK];        // rows of Kt of its state tiles
  int t0, n;                         // the chunk's tokens
};

// grid (B * H, VP / CT), 4 waves: blocks of one (sequence, head) are B * H
// apart, so with B * H a multiple of 8 they share an XCD's L2. Waves 0 and 1
// compute U = U0 - W S0, waves 2 and 3 the outputs; all update the state. The
// next chunks' scratch is loaded while a chunk is computed (AHEAD of them).
template <int DT, int AHEAD>
__global__ __launch_bounds__(BLOCK) void delta_chunk_chain_kernel(
    DeltaScratch s, const int* __restrict__ cu_c, float* __restrict__ S,
    const int* __restrict__ chunk_base, const int* __restrict__ n_chunks,
    const int* __restrict__ slots, const int* __restrict__ pos0,
    float* __restrict__ out, int H, int D, int V, int VP) {
  constexpr int NS = 2, C = 16 * NS, DP = 16 * DT;
  constexpr int NW = DT >= 4 ? DT / 4 : 1;     // state row tiles per wave
  using Frag = ChainFrag<NS, DT, NW>;
  __shared__ __align__(16) float Ss[DP * CS];
  __shared__ __align__(16) float Us[C * CS];
  const int b = blockIdx.x / H, h = blockIdx.x - b * H;
  const int nc = n_chunks[b];
  if (nc <= 0) return;
  const int c0 = blockIdx.y * CT;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int li = lane & 15, quad = lane >> 4;
  const bool is_u = wave < 2;
  const int ta = wave & 1;           // token tile
  const bool has_st = wave * NW < DT;
  const int dt0 = has_st ? wave * NW : 0;           // first state row tile
  const int c = c0 + li;             // this lane's value column
  float* Sh = S + ((int64_t)slots[b] * H + h) * D * V;
  const bool fresh = pos0[b] == 0;
  f32x4 st[NW];
  if (has_st)
#pragma unroll
    for (int i = 0; i < NW; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = (dt0 + i) * 16 + quad * 4 + r;
        const float v =
            !fresh && d < D && c < V ? Sh[(int64_t)d * V + c] : 0.f;
        st[i][r] = v;
        Ss[d * CS + li] = v;
      }
  const int cb = chunk_base[b];
  const float* WQ = is_u ? s.W : s.Q;
  auto load = [&](Frag& f, int k) {
    k = min(k, nc - 1);
    const int64_t ci = (int64_t)(cb + k) * H + h;
    f.t0 = cu_c[cb + k];
    f.n = cu_c[cb + k + 1] - f.t0;
    const float* wq = WQ + ci * C * DP + (ta * DT * 64 + lane) * 4;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
      f.wq[dt] = *reinterpret_cast<const float4*>(wq + dt * 256);
    // (waves 2 and 3 load what they do not use: no branch around a load)
    f.u0 = *reinterpret_cast<const float4*>(
        s.U + ci * C * VP + ((ta * (VP / 16) + blockIdx.y) * 64 + lane) * 4);
#pragma unroll
    for (int i = 0; i < NW; ++i) {
      const float* kp = s.Kt + ci * C * DP +
                        ((dt0 + i) * NS * 64 + lane) * 4;
#pragma unroll
      for (int bb = 0; bb < NS; ++bb)
        f.kt[i][bb] = *reinterpret_cast<const float4*>(kp + bb * 256);
      f.dec[i] = *reinterpret_cast<const float4*>(
          s.dec + ci * DP + (dt0 + i) * 16 + quad * 4);
    }
    const float* bp = s.B + ci * C * C + (ta * NS * 64 + lane) * 4;
#pragma unroll
    for (int bb = 0; bb < NS; ++bb)
      f.b[bb] = *reinterpret_cast<const float4*>(bp + bb * 256);
  };
  auto step = [&](const Frag& f) {
    // ---- W S0 or Q S0, as two sums
    f32x4 p0 = (f32x4){0.f, 0.f, 0.f, 0.f}, p1 = p0;
    float sv[DT][4];
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
#pragma unroll
      for (int e = 0; e < 4; ++e)
        sv[dt][e] = Ss[(dt * 16 + quad * 4 + e) * CS + li];
    __builtin_amdgcn_sched_barrier(0);   // all reads before the products
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      if (dt & 1)
        p1 = mfma4(f.wq[dt], sv[dt][0], sv[dt][1], sv[dt][2], sv[dt][3], p1);
      else
        p0 = mfma4(f.wq[dt], sv[dt][0], sv[dt][1], sv[dt][2], sv[dt][3], p0);
    }
    f32x4 o = p0 + p1;
    if (is_u) {
      float* us = Us + (ta * 16 + quad * 4) * CS + li;
      us[0] = f.u0.x - o[0];
      us[CS] = f.u0.y - o[1];
      us[2 * CS] = f.u0.z - o[2];
      us[3 * CS] = f.u0.w - o[3];
    }
    lds_barrier();
    float uv[NS][4];
#pragma unroll
    for (int bb = 0; bb < NS; ++bb)
#pragma unroll
      for (int e = 0; e < 4; ++e)
        uv[bb][e] = Us[(bb * 16 + quad * 4 + e) * CS + li];
    __builtin_amdgcn_sched_barrier(0);
    // ---- the state after the chunk
    if (has_st)
#pragma unroll
      for (int i = 0; i < NW; ++i) {
        st[i][0] *= f.dec[i].x;
        st[i][1] *= f.dec[i].y;
        st[i][2] *= f.dec[i].z;
        st[i][3] *= f.dec[i].w;
#pragma unroll
        for (int bb = 0; bb < NS; ++bb)
          st[i] = mfma4(f.kt[i][bb], uv[bb][0], uv[bb][1], uv[bb][2],
                        uv[bb][3], st[i]);
        // Ss is read before the barrier above only
#pragma unroll
        for (int r = 0; r < 4; ++r)
          Ss[((dt0 + i) * 16 + quad * 4 + r) * CS + li] = st[i][r];
      }
    // ---- outputs: the chunk's own part
    if (!is_u) {
#pragma unroll
      for (int bb = 0; bb < NS; ++bb) {
        if (bb > ta) continue;
        o = mfma4(f.b[bb], uv[bb][0], uv[bb][1], uv[bb][2], uv[bb][3], o);
      }
      if (c < V)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = ta * 16 + quad * 4 + r;
          if (t < f.n) out[((int64_t)(f.t0 + t) * H + h) * V + c] = o[r];
        }
    }
    lds_barrier();
  };
  lds_barrier();
  // loads are issued unconditionally (past the end: the last chunk again), so
  // that their count is known where they are waited for
  if constexpr (AHEAD == 2) {
    Frag f0, f1, f2;
    load(f0, 0);
    load(f1, 1);
    for (int k = 0;;) {
      load(f2, k + 2);
      step(f0);
      if (++k >= nc) break;
      load(f0, k + 2);
      step(f1);
      if (++k >= nc) break;
      load(f1, k + 2);
      step(f2);
      if (++k >= nc) break;
    }
  } else {
    Frag f0, f1;
    load(f0, 0);
    for (int k = 0;;) {
      load(f1, k + 1);
      step(f0);
      if (++k >= nc) break;
      load(f0, k + 1);
      step(f1);
      if (++k >= nc) break;
    }
  }
  if (has_st)
#pragma unroll
    for (int i = 0; i < NW; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = (dt0 + i) * 16 + quad * 4 + r;
        if (d < D && c < V) Sh[(int64_t)d * V + c] = st[i][r];
      }
}

constexpr size_t LDS_MAX = 64 * 1024 - 1024;

size_t scan_smem(int DR, int R) {
  return sizeof(float) *
         ((size_t)RT * (3 * 4 * (DR + 4) + VT + 1) + (size_t)RT * R);
}

size_t prep_smem(int DT, int R) {
  const size_t C = CHUNK, NS = CHUNK / 16, LS = 16 * DT + 4;
  const size_t a = C * (C + 4), r = C * ((R + 15) / 16 * 16 + 4);
  return sizeof(float) * (3 * C * LS + 3 * NS * LS + (a > r ? a : r));
}

// LDS a block may have on this device (64 KiB where it is not known)
size_t lds_limit() {
  static const size_t lim = [] {
    int dev = 0, v = 0;
    if (hipGetDevice(&dev) != hipSuccess ||
        hipDeviceGetAttribute(&v, hipDeviceAttributeMaxSharedMemoryPerBlock,
                              dev) != hipSuccess ||
        v < 64 * 1024)
      v = 64 * 1024;
    return (size_t)v - 1024;
  }();
  return lim;
}

// row tiles of 16 that cover D: the sizes the chunk kernels are built for
int row_tiles(int D) { return D <= 32 ? 2 : D <= 64 ? 4 : D <= 128 ? 8 : 16; }

template <typename T, int DT, int AHEAD>
void launch_chunks(const T* proj, const DeltaSrc& p, const int* cu_c, int NC,
                   const int* base, const int* cnt, const int* slots,
                   const int* pos0, int B, float* S, const DeltaScratch& s,
                   float* out, int H, int D, int V, int VP,
                   hipStream_t stream) {
  const size_t smem = prep_smem(DT, p.R);
  if (smem > 64 * 1024)
    (void)hipFuncSetAttribute(
        (const void*)delta_chunk_prep_kernel<T, CHUNK / 16, DT>,
        hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
  hipLaunchKernelGGL((delta_chunk_prep_kernel<T, CHUNK / 16, DT>),
                     dim3(NC, H), dim3(BLOCK), smem, stream, proj, p, cu_c, s,
                     H, D, V, VP);
  hipLaunchKernelGGL((delta_chunk_chain_kernel<DT, AHEAD>),
                     dim3(B * H, VP / CT), dim3(BLOCK), 0, stream, s, cu_c,
                     S, base, cnt, slots, pos0, out, H, D, V, VP);
}

template <typename T>
void chunks_any(const T* proj, const DeltaSrc& p, const int* cu_c, int NC,
                const int* base, const int* cnt, const int* slots,
                const int* pos0, int B, float* S, const DeltaScratch& s,
                float* out, int H, int D, int V, int VP, hipStream_t stream) {
#define TL_DC(DT, AHEAD)                                                     \
  launch_chunks<T, DT, AHEAD>(proj, p, cu_c, NC, base, cnt, slots, pos0, B, \
                              S, s, out, H, D, V, VP, stream)
  const int dt = row_tiles(D);
  if (dt <= 2) TL_DC(2, 2);
  else if (dt <= 4) TL_DC(4, 2);
  else if (dt <= 8) TL_DC(8, 1);
  else TL_DC(16, 1);
#undef TL_DC
}

}  // namespace

extern "C" {

int tl_delta_chunk_tokens() { return CHUNK; }

// 1 if the chunk form serves the shape
int tl_delta_chunks_ok(int D, int R) {
  if (D < 1 || D > 256 || R < 1) return 0;
  return prep_smem(row_tiles(D), R) <= lds_limit() ? 1 : 0;
}

int tl_delta_row_pad(int D) { return 16 * row_tiles(D); }
int tl_delta_col_pad(int V) { return (V + CT - 1) / CT * CT; }

// returns 0 on success, 1 if the shape is outside what the kernels serve.
// Scratch sizes: see DeltaScratch (W, Q, Kt, B, U, dec per chunk and head)
int tl_delta_chunks(const void* x, int ldx, int q_off, int k_off, int v_off,
                    const void* proj, int ldr, int r_off, int R,
                    const void* b, int ldb, int b_off, const void* a2t,
                    const void* dt_bias, const void* A_log, float qscale,
                    void* S, const void* cu_c, int NC, const void* base,
                    const void* cnt, const void* slots, const void* pos0,
                    int B, void* W, void* Q, void* Kt, void* Bm, void* U,
                    void* dec, void* out, int H, int G, int D, int V,
                    int is_f32, hipStream_t stream) {
  if (!tl_delta_chunks_ok(D, R) || H <= 0 || V <= 0 || G <= 0 ||
      H % G != 0)
    return 1;
  if (NC <= 0 || B <= 0) return 0;
  DeltaSrc p{(const float*)x, ldx, q_off, k_off, v_off, ldr, r_off, R,
             (const float*)b, ldb, b_off, (const float*)a2t,
             (const float*)dt_bias, (const float*)A_log, qscale, H / G};
  DeltaScratch s{(float*)W, (float*)Q, (float*)Kt,
                 (float*)Bm, (float*)U, (float*)dec};
  const int VP = tl_delta_col_pad(V);
  if (is_f32)
    chunks_any<float>((const float*)proj, p, (const int*)cu_c, NC,
                      (const int*)base, (const int*)cnt, (const int*)slots,
                      (const int*)pos0, B, (float*)S, s, (float*)out, H, D, V,
                      VP, stream);
  else
    chunks_any<bf16>((const bf16*)proj, p, (const int*)cu_c, NC,
                     (const int*)base, (const int*)cnt, (const int*)slots,
                     (const int*)pos0, B, (float*)S, s, (float*)out, H, D, V,
                     VP, stream);
  return 0;
}

// returns 0 on success, 1 if the launch cannot be made
int tl_delta_scan(const void* x, int ldx, int q_off, int k_off, int v_off,
                  const void* proj, int ldr, int r_off, int R, const void* b,
                  int ldb, int b_off, const void* a2t, const void* dt_bias,
                  const void* A_log, float qscale, void* S, const void* cu,
                  const void* slots, const void* pos0, void* out, int B,
                  int H, int G, int D, int V, int is_f32,
                  hipStream_t stream) {
  if (B <= 0 || H <= 0 || G <= 0 || H % G != 0 || D <= 0 || V <= 0 || R <= 0)
    return 1;
  DeltaSrc p{(const float*)x, ldx, q_off, k_off, v_off, ldr, r_off, R,
             (const float*)b, ldb, b_off, (const float*)a2t,
             (const float*)dt_bias, (const float*)A_log, qscale, H / G};
  dim3 grid(B, H, (V + VT - 1) / VT), block(BLOCK);
#define TL_DS(TT, DR)                                                       \
  hipLaunchKernelGGL((delta_scan_kernel<TT, DR>), grid, block,              \
                     scan_smem(DR, R), stream, (const TT*)proj, p,          \
                     (float*)S, (const int*)cu, (const int*)slots,          \
                     (const int*)pos0, (float*)out, H, D, V)
#define TL_DS_T(DR)                                     \
  if (D <= 4 * DR && scan_smem(DR, R) <= LDS_MAX) {     \
    if (is_f32) TL_DS(float, DR);                       \
    else TL_DS(bf16, DR);                               \
    return 0;                                           \
  }
  TL_DS_T(8)
  TL_DS_T(16)
  TL_DS_T(32)
  TL_DS_T(64)
#undef TL_DS_T
#undef TL_DS
  const size_t gsmem = sizeof(float) * 3 * (size_t)D;
  if (gsmem > LDS_MAX) return 1;
  dim3 g2(B, H);
  if (is_f32)
    hipLaunchKernelGGL(delta_scan_generic_kernel<float>, g2, block, gsmem,
                       stream, (const float*)proj, p, (float*)S,
                       (const int*)cu, (const int*)slots, (const int*)pos0,
                       (float*)out, H, D, V);
  else
    hipLaunchKernelGGL(delta_scan_generic_kernel<bf16>, g2, block, gsmem,
                       stream, (const bf16*)proj, p, (float*)S,
                       (const int*)cu, (const int*)slots, (const int*)pos0,
                       (float*)out, H, D, V);
  return 0;
}

}  // extern "C"
