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
// Long prompt portions take the chunk form: chunks of C = 16 * NS tokens in
// NS tiles of 16. With L_t the running sum of log g inside the chunk,
//     A_ts = beta_t sum_d k_td k_sd e^(L_td - L_sd)               (s < t)
//     (I + A) U = diag(beta) V - diag(beta) [K e^L] S0
//     O  = [Q e^L] S0 + B U,  B_ts = sum_d q_td k_sd e^(L_td - L_sd)  (s <= t)
//     S1 = e^(L_C) S0 + [K e^(L_C - L)]^T U
// tl_delta_chunk_prep computes, per chunk and head, W = (I + A)^-1 diag(beta)
// [K e^L] and U0 = (I + A)^-1 diag(beta) V by block forward substitution (the
// 16 x 16 diagonal blocks are inverted), B, [Q e^L], [K e^(L_C - L)]^T and
// e^(L_C). tl_delta_chunk_chain then walks a sequence's chunks with
// U = U0 - W S0; one block per (sequence, head, 32 value columns).
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
constexpr int CT = 32;              // value columns per block of the chain
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
    // decays, spread over the block
    for (int i = threadIdx.x; i < nt * 4 * DR; i += BLOCK) {
      const int tt = i / (4 * DR), d = i - tt * (4 * DR);
      float a = 1.f;
      if (d < D) {
        const int hd = h * D + d;
        float z = p.dt_bias[hd];
        for (int r = 0; r < p.R; ++r)
          z += rs[tt * p.R + r] * p.a2t[(int64_t)r * H * D + hd];
        a = expf(ea * softplus_f(z));
      }
      gs[tt * DP + (d / DR) * GS + d % DR] = a;
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

// grid (chunks, H)
template <typename T, int NS, int DT>
__global__ __launch_bounds__(BLOCK) void delta_chunk_prep_kernel(
    const T* __restrict__ proj, DeltaSrc p, const int* __restrict__ cu_c,
    DeltaScratch s, int H, int D, int V, int VP) {
  constexpr int C = 16 * NS, DP = 16 * DT;
  constexpr int LS = DP + 4, AS = C + 4;
  extern __shared__ __align__(16) float lds[];
  __shared__ int far[NS];
  __shared__ float qn[C], kn[C], bt[C];
  float* L = lds;                  // [C][LS] running logs inside a tile
  float* tot = L + C * LS;         // [NS][LS]
  float* A = tot + NS * LS;        // [C][AS]; first the low-rank rows [R][C]
  const int ch = blockIdx.x, h = blockIdx.y, hq = h / p.rep;
  const int t0 = cu_c[ch], n = cu_c[ch + 1] - t0;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int li = lane & 15, quad = lane >> 4;
  const float* qh = p.x + (int64_t)t0 * p.ldx + p.q_off + hq * D;
  const float* kh = p.x + (int64_t)t0 * p.ldx + p.k_off + hq * D;
  const float* vh = p.x + (int64_t)t0 * p.ldx + p.v_off + h * V;
  const int64_t ci = (int64_t)ch * H + h;

  // ---- decays: running sums of log g inside each tile, tile totals
  if (threadIdx.x < NS) far[threadIdx.x] = 0;
  for (int i = threadIdx.x; i < C * p.R; i += BLOCK) {
    const int t = i / p.R, r = i - t * p.R;
    A[r * C + t] =
        t < n ? ldf<T>(proj + (int64_t)(t0 + t) * p.ldr + p.r_off + r) : 0.f;
  }
  // norms and step sizes meanwhile: four tokens per wave and step
  for (int t = wave * 4 + quad; t < C; t += 16) {
    float sq = 0.f, sk = 0.f;
    if (t < n)
      for (int d = li; d < D; d += 16) {
        const float q = qh[(int64_t)t * p.ldx + d];
        const float k = kh[(int64_t)t * p.ldx + d];
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
      bt[t] = t < n ? 1.f / (1.f + expf(-p.b[(int64_t)(t0 + t) * p.ldb +
                                             p.b_off + h]))
                    : 0.f;
    }
  }
  __syncthreads();
  const float ea = -expf(p.A_log[h]);
  for (int i = threadIdx.x; i < NS * DP; i += BLOCK) {
    const int a = i / DP, d = i - a * DP;
    const int hd = h * D + d;
    float z[16];
    const float bz = d < D ? p.dt_bias[hd] : 0.f;
#pragma unroll
    for (int t = 0; t < 16; ++t) z[t] = bz;
    if (d < D)
      for (int r = 0; r < p.R; ++r) {
        const float w = p.a2t[(int64_t)r * H * D + hd];
        const float4* rr = reinterpret_cast<const float4*>(A + r * C + a * 16);
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
      if (d < D && a * 16 + t < n)
        run += fmaxf(ea * softplus_f(z[t]), LOG_FLOOR);
      L[(a * 16 + t) * LS + d] = run;
    }
    tot[a * LS + d] = run;
    if (run < -LOG_RANGE) far[a] = 1;      // same value from every writer
  }
  __syncthreads();

  // ---- A (strictly lower, times beta) into LDS, B to memory, by tiles
  float* Bc = s.B + ci * C * C;
  for (int u = wave; u < NS * NS; u += 4) {
    const int a = u / NS, b = u - a * NS;
    f32x4 ak = (f32x4){0.f, 0.f, 0.f, 0.f}, aq = ak;
    if (b <= a && a * 16 < n) {
      if (a == b && far[a]) {
        // strong decay inside the tile: every score on its own
        const int j = a * 16 + li;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int i = a * 16 + quad * 4 + r;
          float sk = 0.f, sq = 0.f;
          if (j <= i && i < n)
            for (int d = 0; d < D; ++d) {
              const float w = kh[(int64_t)j * p.ldx + d] *
                              expf(L[i * LS + d] - L[j * LS + d]);
              sk += kh[(int64_t)i * p.ldx + d] * w;
              sq += qh[(int64_t)i * p.ldx + d] * w;
            }
          const float f = kn[j];
          ak[r] = sk * f * kn[i];
          aq[r] = sq * f * qn[i];
        }
      } else {
        const int i = a * 16 + li, j = b * 16 + li;
        const float fk = kn[i], fq = qn[i], fj = kn[j];
#pragma unroll 2
        for (int dt = 0; dt < DT; ++dt) {
          const int d = dt * 16 + quad * 4;
          float q[4], ki[4], kj[4];
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const bool in = d + e < D;
            q[e] = in && i < n ? qh[(int64_t)i * p.ldx + d + e] : 0.f;
            ki[e] = in && i < n ? kh[(int64_t)i * p.ldx + d + e] : 0.f;
            kj[e] = in && j < n ? kh[(int64_t)j * p.ldx + d + e] : 0.f;
          }
          const float4 x = *reinterpret_cast<const float4*>(L + i * LS + d);
          const float4 y = *reinterpret_cast<const float4*>(L + j * LS + d);
          float ei[4] = {x.x, x.y, x.z, x.w};
          float ej[4] = {-y.x, -y.y, -y.z, -y.w};
          if (a != b) {
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              ej[e] += tot[b * LS + d + e];
              for (int m = b + 1; m < a; ++m) ei[e] += tot[m * LS + d + e];
            }
          }
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const float wi = expf(ei[e]), wj = kj[e] * fj * expf(ej[e]);
            ak = __builtin_amdgcn_mfma_f32_16x16x4f32(ki[e] * fk * wi, wj, ak,
                                                      0, 0, 0);
            aq = __builtin_amdgcn_mfma_f32_16x16x4f32(q[e] * fq * wi, wj, aq,
                                                      0, 0, 0);
          }
        }
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = a * 16 + quad * 4 + r, j = b * 16 + li;
      A[i * AS + j] = j < i ? ak[r] * bt[i] : 0.f;
      Bc[i * C + j] = j <= i ? aq[r] : 0.f;
    }
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
    f32x4 X[NS];
    float before = 0.f;              // sum of the earlier tiles' logs
#pragma unroll
    for (int a = 0; a < NS; ++a) {
      f32x4 y;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = a * 16 + quad * 4 + r;
        float v = 0.f;
        if (i < n) {
          if (isw) {
            if (col < D)
              v = kh[(int64_t)i * p.ldx + col] * kn[i] *
                  expf(before + L[i * LS + col]);
          } else if (col < V) {
            v = vh[(int64_t)i * p.ldx + col];
          }
        }
        y[r] = v * bt[i];
      }
      if (isw) before += tot[a * LS + col];
      for (int b = 0; b < a; ++b) {
        const float4 f = *reinterpret_cast<const float4*>(
            A + (a * 16 + li) * AS + b * 16 + quad * 4);
        y = __builtin_amdgcn_mfma_f32_16x16x4f32(-f.x, X[b][0], y, 0, 0, 0);
        y = __builtin_amdgcn_mfma_f32_16x16x4f32(-f.y, X[b][1], y, 0, 0, 0);
        y = __builtin_amdgcn_mfma_f32_16x16x4f32(-f.z, X[b][2], y, 0, 0, 0);
        y = __builtin_amdgcn_mfma_f32_16x16x4f32(-f.w, X[b][3], y, 0, 0, 0);
      }
      const float4 f = *reinterpret_cast<const float4*>(
          A + (a * 16 + li) * AS + a * 16 + quad * 4);
      f32x4 z = (f32x4){0.f, 0.f, 0.f, 0.f};
      z = __builtin_amdgcn_mfma_f32_16x16x4f32(f.x, y[0], z, 0, 0, 0);
      z = __builtin_amdgcn_mfma_f32_16x16x4f32(f.y, y[1], z, 0, 0, 0);
      z = __builtin_amdgcn_mfma_f32_16x16x4f32(f.z, y[2], z, 0, 0, 0);
      z = __builtin_amdgcn_mfma_f32_16x16x4f32(f.w, y[3], z, 0, 0, 0);
      X[a] = z;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = a * 16 + quad * 4 + r;
        if (isw) Wc[i * DP + col] = z[r];
        else Uc[i * VP + col] = z[r];
      }
    }
  }

  // ---- q e^L, (k e^(L_C - L))^T and e^(L_C)
  float* Qc = s.Q + ci * C * DP;
  for (int i = threadIdx.x; i < C * DP; i += BLOCK) {
    const int t = i / DP, d = i - t * DP, a = t >> 4;
    float v = 0.f;
    if (t < n && d < D) {
      float e = L[t * LS + d];
      for (int m = 0; m < a; ++m) e += tot[m * LS + d];
      v = qh[(int64_t)t * p.ldx + d] * qn[t] * expf(e);
    }
    Qc[i] = v;
  }
  float* Kc = s.Kt + ci * C * DP;
  for (int i = threadIdx.x; i < C * DP; i += BLOCK) {
    const int d = i / C, t = i - d * C, a = t >> 4;
    float v = 0.f;
    if (t < n && d < D) {
      float e = tot[a * LS + d] - L[t * LS + d];
      for (int m = a + 1; m < NS; ++m) e += tot[m * LS + d];
      v = kh[(int64_t)t * p.ldx + d] * kn[t] * expf(e);
    }
    Kc[i] = v;
  }
  for (int d = threadIdx.x; d < DP; d += BLOCK) {
    float e = 0.f;
#pragma unroll
    for (int m = 0; m < NS; ++m) e += tot[m * LS + d];
    s.dec[ci * DP + d] = expf(e);
  }
}

// grid (B * H, VP / CT): blocks of one (sequence, head) are B * H apart, so
// with B * H a multiple of 8 they share an XCD's L2
template <int NS, int DT>
__global__ __launch_bounds__(BLOCK) void delta_chunk_chain_kernel(
    DeltaScratch s, const int* __restrict__ cu_c, float* __restrict__ S,
    const int* __restrict__ chunk_base, const int* __restrict__ n_chunks,
    const int* __restrict__ slots, const int* __restrict__ pos0,
    float* __restrict__ out, int H, int D, int V, int VP) {
  constexpr int C = 16 * NS, DP = 16 * DT;
  // units of work per wave: token tile x column tile (NS * 2 over 4 waves),
  // state row tile x column tile (DT * 2 over 4 waves)
  constexpr int NU = NS * 2 / 4, NW = DT * 2 / 4;
  __shared__ __align__(16) float Ss[DP * CS];
  __shared__ __align__(16) float Us[C * CS];
  const int b = blockIdx.x / H, h = blockIdx.x - b * H;
  const int nc = n_chunks[b];
  if (nc <= 0) return;
  const int c0 = blockIdx.y * CT;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int li = lane & 15, quad = lane >> 4;
  float* Sh = S + ((int64_t)slots[b] * H + h) * D * V;
  const bool fresh = pos0[b] == 0;
  f32x4 st[NW];
#pragma unroll
  for (int i = 0; i < NW; ++i) {
    const int w = wave * NW + i, dt = w >> 1, x = w & 1;
    const int c = c0 + x * 16 + li;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = dt * 16 + quad * 4 + r;
      const float v =
          !fresh && d < D && c < V ? Sh[(int64_t)d * V + c] : 0.f;
      st[i][r] = v;
      Ss[d * CS + x * 16 + li] = v;
    }
  }
  __syncthreads();
  const int cb = chunk_base[b];
  for (int k = 0; k < nc; ++k) {
    const int ch = cb + k;
    const int64_t ci = (int64_t)ch * H + h;
    const int t0 = cu_c[ch], n = cu_c[ch + 1] - t0;
    // ---- U = U0 - W S0 and the carried part of the outputs
    f32x4 uo[NU], oo[NU];
#pragma unroll
    for (int i = 0; i < NU; ++i) {
      const int w = wave * NU + i, a = w >> 1, x = w & 1;
      const float* U0 = s.U + (ci * C + a * 16 + quad * 4) * VP + c0 +
                        x * 16 + li;
#pragma unroll
      for (int r = 0; r < 4; ++r) uo[i][r] = U0[(int64_t)r * VP];
      oo[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
#pragma unroll
      for (int i = 0; i < NU; ++i) {
        const int w = wave * NU + i, a = w >> 1, x = w & 1;
        const int64_t ro = (ci * C + a * 16 + li) * DP + dt * 16 + quad * 4;
        const float4 wv = *reinterpret_cast<const float4*>(s.W + ro);
        const float4 qv = *reinterpret_cast<const float4*>(s.Q + ro);
        const float* sp = Ss + (dt * 16 + quad * 4) * CS + x * 16 + li;
        const float s0 = sp[0], s1 = sp[CS], s2 = sp[2 * CS], s3 = sp[3 * CS];
        uo[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(-wv.x, s0, uo[i], 0, 0, 0);
        oo[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(qv.x, s0, oo[i], 0, 0, 0);
        uo[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(-wv.y, s1, uo[i], 0, 0, 0);
        oo[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(qv.y, s1, oo[i], 0, 0, 0);
        uo[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(-wv.z, s2, uo[i], 0, 0, 0);
        oo[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(qv.z, s2, oo[i], 0, 0, 0);
        uo[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(-wv.w, s3, uo[i], 0, 0, 0);
        oo[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(qv.w, s3, oo[i], 0, 0, 0);
      }
    }
#pragma unroll
    for (int i = 0; i < NU; ++i) {
      const int w = wave * NU + i, a = w >> 1, x = w & 1;
#pragma unroll
      for (int r = 0; r < 4; ++r)
        Us[(a * 16 + quad * 4 + r) * CS + x * 16 + li] = uo[i][r];
    }
    __syncthreads();
    // ---- outputs: the chunk's own part
#pragma unroll
    for (int i = 0; i < NU; ++i) {
      const int w = wave * NU + i, a = w >> 1, x = w & 1;
      const float* Bp = s.B + (ci * C + a * 16 + li) * C + quad * 4;
#pragma unroll
      for (int bb = 0; bb < NS; ++bb) {
        if (bb > a) continue;
        const float4 f = *reinterpret_cast<const float4*>(Bp + bb * 16);
        const float* up = Us + (bb * 16 + quad * 4) * CS + x * 16 + li;
        oo[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.x, up[0], oo[i], 0, 0, 0);
        oo[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.y, up[CS], oo[i], 0, 0, 0);
        oo[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.z, up[2 * CS], oo[i], 0, 0, 0);
        oo[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.w, up[3 * CS], oo[i], 0, 0, 0);
      }
      const int c = c0 + x * 16 + li;
      if (c < V)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = a * 16 + quad * 4 + r;
          if (t < n) out[((int64_t)(t0 + t) * H + h) * V + c] = oo[i][r];
        }
    }
    // ---- the state after the chunk
#pragma unroll
    for (int i = 0; i < NW; ++i) {
      const int w = wave * NW + i, dt = w >> 1, x = w & 1;
      const float4 de =
          *reinterpret_cast<const float4*>(s.dec + ci * DP + dt * 16 + quad * 4);
      st[i][0] *= de.x;
      st[i][1] *= de.y;
      st[i][2] *= de.z;
      st[i][3] *= de.w;
      const float* Kp = s.Kt + (ci * DP + dt * 16 + li) * C + quad * 4;
#pragma unroll
      for (int bb = 0; bb < NS; ++bb) {
        const float4 f = *reinterpret_cast<const float4*>(Kp + bb * 16);
        const float* up = Us + (bb * 16 + quad * 4) * CS + x * 16 + li;
        st[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.x, up[0], st[i], 0, 0, 0);
        st[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.y, up[CS], st[i], 0, 0, 0);
        st[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.z, up[2 * CS], st[i], 0, 0, 0);
        st[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.w, up[3 * CS], st[i], 0, 0, 0);
      }
      // Ss is read before the barrier above only
#pragma unroll
      for (int r = 0; r < 4; ++r)
        Ss[(dt * 16 + quad * 4 + r) * CS + x * 16 + li] = st[i][r];
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < NW; ++i) {
    const int w = wave * NW + i, dt = w >> 1, x = w & 1;
    const int c = c0 + x * 16 + li;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = dt * 16 + quad * 4 + r;
      if (d < D && c < V) Sh[(int64_t)d * V + c] = st[i][r];
    }
  }
}

constexpr size_t LDS_MAX = 64 * 1024 - 1024;

size_t scan_smem(int DR, int R) {
  return sizeof(float) *
         ((size_t)RT * (3 * 4 * (DR + 4) + VT + 1) + (size_t)RT * R);
}

size_t prep_smem(int NS, int DT, int R) {
  const size_t C = 16 * NS, LS = 16 * DT + 4;
  const size_t a = C * (C + 4), r = C * R;
  return sizeof(float) * (C * LS + NS * LS + (a > r ? a : r));
}

// row tiles of 16 that cover D: the sizes the chunk kernels are built for
int row_tiles(int D) { return D <= 32 ? 2 : D <= 64 ? 4 : D <= 128 ? 8 : 16; }

template <typename T, int NS, int DT>
void launch_chunks(const T* proj, const DeltaSrc& p, const int* cu_c, int NC,
                   const int* base, const int* cnt, const int* slots,
                   const int* pos0, int B, float* S, const DeltaScratch& s,
                   float* out, int H, int D, int V, int VP,
                   hipStream_t stream) {
  hipLaunchKernelGGL((delta_chunk_prep_kernel<T, NS, DT>), dim3(NC, H),
                     dim3(BLOCK), prep_smem(NS, DT, p.R), stream, proj, p,
                     cu_c, s, H, D, V, VP);
  hipLaunchKernelGGL((delta_chunk_chain_kernel<NS, DT>), dim3(B * H, VP / CT),
                     dim3(BLOCK), 0, stream, s, cu_c, S, base, cnt, slots,
                     pos0, out, H, D, V, VP);
}

template <typename T>
void chunks_any(const T* proj, const DeltaSrc& p, const int* cu_c, int NC,
                const int* base, const int* cnt, const int* slots,
                const int* pos0, int B, float* S, const DeltaScratch& s,
                float* out, int H, int D, int V, int VP, int C,
                hipStream_t stream) {
#define TL_DC(NS, DT)                                                       \
  launch_chunks<T, NS, DT>(proj, p, cu_c, NC, base, cnt, slots, pos0, B, S, \
                           s, out, H, D, V, VP, stream)
  const int dt = row_tiles(D);
  if (C == 64) {
    if (dt <= 2) TL_DC(4, 2);
    else TL_DC(4, 4);
  } else {
    if (dt <= 2) TL_DC(2, 2);
    else if (dt <= 4) TL_DC(2, 4);
    else if (dt <= 8) TL_DC(2, 8);
    else TL_DC(2, 16);
  }
#undef TL_DC
}

}  // namespace

extern "C" {

// 1 if the chunk form serves the shape with chunks of C tokens
int tl_delta_chunks_ok(int D, int R, int C) {
  if (C != 64 && C != 32) return 0;
  if (D < 1 || D > 256 || R < 1 || (C == 64 && D > 64)) return 0;
  return prep_smem(C / 16, row_tiles(D), R) <= LDS_MAX ? 1 : 0;
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
                    void* dec, void* out, int H, int G, int D, int V, int C,
                    int is_f32, hipStream_t stream) {
  if (!tl_delta_chunks_ok(D, R, C) || H <= 0 || V <= 0 || G <= 0 ||
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
                      VP, C, stream);
  else
    chunks_any<bf16>((const bf16*)proj, p, (const int*)cu_c, NC,
                     (const int*)base, (const int*)cnt, (const int*)slots,
                     (const int*)pos0, B, (float*)S, s, (float*)out, H, D, V,
                     VP, C, stream);
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
