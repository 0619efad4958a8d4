// Row-wise kernels of the post-norm layered family (gfx950).
//
// The residual X is fp32 and every sublayer's output y is normalised
// BEFORE it is added:  X <- X + y / rms(y) * g,  g = w or 1 + w.
// tl_postnorm_add does the row statistic, the scaled add and the cast of
// the new residual to the serving dtype (the next sublayer's GEMM input)
// in one kernel: y is read twice (the second time from cache), X makes one
// round trip. tl_rms_scale is the plain / gated RMS scaling (final norm;
// read-out norm of a linear-attention mixer with its sigmoid gate), tl_gelu
// the exact or tanh-form GELU with an optional gathered per-token factor,
// tl_soft_cap the logit cap. Statistics and activations are fp32.
//
// Pre-norm layers use tl_add_rms: the previous sublayer's output is added
// to the fp32 residual and the NEXT sublayer's input, rms(X) * w, is written
// in the serving dtype by the same kernel (X <- X + y;  h = X / rms(X) * w).
// A gated residual multiplies y element by element by the sigmoid of columns
// of the sublayer's own projection in the same pass. Rows of a multiple of 4
// columns are held in registers between the statistic and the scaling.
// tl_act_gate is the gated feed-forward's activation on a fused [gate | up]
// projection: act(gate) * up, act = gelu (erf / tanh form), silu or relu, or
// the clamped swish. A residual sum may have up to three terms, each with a
// factor (sublayers side by side). tl_head_rms_gate is the read-out norm of a
// linear-attention mixer whose heads are normed on their own:
// x_h / rms(x_h) * w [* silu(gate) | sigmoid(gate)].

#include "common.hpp"

namespace {

constexpr int BLOCK = 256;
constexpr int NW = BLOCK / WAVE_SIZE;

template <typename T> DEVINLINE float ldf(const T* p, int64_t i);
template <> DEVINLINE float ldf<float>(const float* p, int64_t i) { return p[i]; }
template <> DEVINLINE float ldf<bf16>(const bf16* p, int64_t i) { return bf2f(p[i]); }
template <typename T> DEVINLINE void stf(T* p, int64_t i, float v);
template <> DEVINLINE void stf<float>(float* p, int64_t i, float v) { p[i] = v; }
template <> DEVINLINE void stf<bf16>(bf16* p, int64_t i, float v) { p[i] = f2bf(v); }

DEVINLINE float gelu_f(float z, int tanh_form) {
  if (tanh_form)
    return 0.5f * z *
           (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
  return 0.5f * z * (1.f + erff(z * 0.7071067811865476f));
}

// one block per row
template <typename T>
__global__ __launch_bounds__(BLOCK) void postnorm_add_kernel(
    float* __restrict__ X, const T* __restrict__ y,
    const float* __restrict__ w, T* __restrict__ h, int W, float eps,
    int one_plus) {
  __shared__ float red[NW];
  const int64_t row = blockIdx.x;
  const T* yr = y + row * W;
  float ss = 0.f;
  for (int c = threadIdx.x; c < W; c += BLOCK) {
    const float v = ldf<T>(yr, c);
    ss += v * v;
  }
  const float tot = block_reduce_sum<NW>(ss, red);
  const float rn = 1.0f / sqrtf(tot / (float)W + eps);
  float* xr = X + row * W;
  for (int c = threadIdx.x; c < W; c += BLOCK) {
    const float g = one_plus ? 1.f + w[c] : w[c];
    const float v = xr[c] + ldf<T>(yr, c) * rn * g;
    xr[c] = v;
    if (h) stf<T>(h, row * W + c, v);
  }
}

// further terms of a residual sum beside the first, and every term's factor
template <typename T>
struct AddMore {
  const T* y1;
  const T* y2;
  float s0, s1, s2;
};

// y[c] [* sigmoid(gate[c])]
template <typename T>
DEVINLINE float gated(const T* y, const T* gate, int64_t c) {
  const float v = ldf<T>(y, c);
  return gate ? v / (1.f + expf(-ldf<T>(gate, c))) : v;
}

// X += sum of the given terms; h = X / rms(X) * w in the serving dtype (no w:
// no h)
template <typename T>
__global__ __launch_bounds__(BLOCK) void add_rms_kernel(
    float* __restrict__ X, const T* __restrict__ y,
    const float* __restrict__ w, T* __restrict__ h, int W, float eps,
    float x_scale, const T* __restrict__ gate, int ldg, AddMore<T> more) {
  __shared__ float red[NW];
  const int64_t row = blockIdx.x;
  float* xr = X + row * W;
  const T* yr = y ? y + row * W : nullptr;
  const T* gr = gate ? gate + row * ldg : nullptr;
  float ss = 0.f;
  for (int c = threadIdx.x; c < W; c += BLOCK) {
    float v = xr[c] * x_scale;
    if (y) v += more.s0 * gated<T>(yr, gr, c);
    if (more.y1) v += more.s1 * ldf<T>(more.y1, row * W + c);
    if (more.y2) v += more.s2 * ldf<T>(more.y2, row * W + c);
    if (y || x_scale != 1.f) xr[c] = v;
    ss += v * v;
  }
  if (!w) return;                 // the residual add alone
  const float tot = block_reduce_sum<NW>(ss, red);
  const float rn = 1.0f / sqrtf(tot / (float)W + eps);
  // a thread reads back only what it wrote itself
  for (int c = threadIdx.x; c < W; c += BLOCK)
    stf<T>(h, row * W + c, xr[c] * rn * w[c]);
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
DEVINLINE void st4(float* p, const float (&v)[4]) {
  *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
}
DEVINLINE void st4(bf16* p, const float (&v)[4]) {
  bf16x4 o;
#pragma unroll
  for (int e = 0; e < 4; ++e) o.v[e] = f2bf(v[e]);
  *reinterpret_cast<bf16x4*>(p) = o;
}

// the same for W a multiple of 4 and W <= 4 * BLOCK * NV: the row stays in
// registers between the sum and the scaling
template <typename T, int NV>
__global__ __launch_bounds__(BLOCK) void add_rms_vec_kernel(
    float* __restrict__ X, const T* __restrict__ y,
    const float* __restrict__ w, T* __restrict__ h, int W, float eps,
    float x_scale, const T* __restrict__ gate, int ldg, AddMore<T> more) {
  __shared__ float red[NW];
  const int64_t row = blockIdx.x;
  float* xr = X + row * W;
  const T* yr = y ? y + row * W : nullptr;
  const T* gr = gate ? gate + row * ldg : nullptr;
  float v[NV][4];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = (k * BLOCK + threadIdx.x) * 4;
    if (c < W) {
      ld4(xr + c, v[k]);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[k][e] *= x_scale;
      if (y) {
        float u[4];
        ld4(yr + c, u);
        if (gate) {
          float g[4];
          ld4(gr + c, g);
#pragma unroll
          for (int e = 0; e < 4; ++e) u[e] = u[e] / (1.f + expf(-g[e]));
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) v[k][e] += more.s0 * u[e];
      }
      if (more.y1) {
        float u[4];
        ld4(more.y1 + row * W + c, u);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[k][e] += more.s1 * u[e];
      }
      if (more.y2) {
        float u[4];
        ld4(more.y2 + row * W + c, u);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[k][e] += more.s2 * u[e];
      }
      if (y || x_scale != 1.f) st4(xr + c, v[k]);
#pragma unroll
      for (int e = 0; e < 4; ++e) ss += v[k][e] * v[k][e];
    }
  }
  if (!w) return;
  const float tot = block_reduce_sum<NW>(ss, red);
  const float rn = 1.0f / sqrtf(tot / (float)W + eps);
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = (k * BLOCK + threadIdx.x) * 4;
    if (c < W) {
      float g[4];
      ld4(w + c, g);
#pragma unroll
      for (int e = 0; e < 4; ++e) g[e] *= v[k][e] * rn;
      st4(h + row * W + c, g);
    }
  }
}

template <typename T>
void launch_add_rms(float* X, const T* y, const float* w, T* h, int64_t rows,
                    int W, float eps, float x_scale, const T* gate, int ldg,
                    AddMore<T> more, bool vec, hipStream_t stream) {
  dim3 grid((unsigned)rows), block(BLOCK);
#define TL_AR(NV)                                                           \
  hipLaunchKernelGGL((add_rms_vec_kernel<T, NV>), grid, block, 0, stream, X, \
                     y, w, h, W, eps, x_scale, gate, ldg, more)
  const int nv = (W / 4 + BLOCK - 1) / BLOCK;
  if (vec && nv <= 1) TL_AR(1);
  else if (vec && nv <= 2) TL_AR(2);
  else if (vec && nv <= 4) TL_AR(4);
  else if (vec && nv <= 8) TL_AR(8);
  else
    hipLaunchKernelGGL(add_rms_kernel<T>, grid, block, 0, stream, X, y, w, h,
                       W, eps, x_scale, gate, ldg, more);
#undef TL_AR
}

// a gated feed-forward's activation of (gate g, up u): 0 erf GELU, 1
// tanh-form GELU, 2 silu, 3 relu, times u; 4 the clamped swish, with g <=
// lim and |u| <= lim, g sigmoid(alpha g) (u + 1)
DEVINLINE float pair_act(float g, float u, int act, float lim, float alpha) {
  if (act == 4) {
    g = fminf(g, lim);
    u = fminf(fmaxf(u, -lim), lim);
    return g / (1.f + expf(-alpha * g)) * (u + 1.f);
  }
  if (act == 3) return fmaxf(g, 0.f) * u;
  if (act == 2) return g / (1.f + expf(-g)) * u;
  return gelu_f(g, act) * u;
}

// out[r][c] = pair_act(p[r][c], p[r][N + c]) on rows of stride ld
template <typename T>
__global__ __launch_bounds__(BLOCK) void act_gate_kernel(
    const T* __restrict__ p, int64_t ld, T* __restrict__ out, int64_t n,
    int N, int act, float lim, float alpha) {
  for (int64_t i = (int64_t)blockIdx.x * BLOCK + threadIdx.x; i < n;
       i += (int64_t)gridDim.x * BLOCK) {
    const int64_t r = i / N;
    const int c = (int)(i - r * N);
    const T* row = p + r * ld;
    stf<T>(out, i,
           pair_act(ldf<T>(row, c), ldf<T>(row, N + c), act, lim, alpha));
  }
}

// bf16, N, the stride and the first column multiples of 8: 16-byte accesses
__global__ __launch_bounds__(BLOCK) void act_gate_vec8_kernel(
    const bf16x8* __restrict__ p, int64_t ld8, bf16x8* __restrict__ out,
    int64_t n8, int N8, int act, float lim, float alpha) {
  for (int64_t i = (int64_t)blockIdx.x * BLOCK + threadIdx.x; i < n8;
       i += (int64_t)gridDim.x * BLOCK) {
    const int64_t r = i / N8;
    const int c = (int)(i - r * N8);
    const bf16x8 a = p[r * ld8 + c], b = p[r * ld8 + N8 + c];
    bf16x8 o;
#pragma unroll
    for (int e = 0; e < 8; ++e)
      o.v[e] = f2bf(pair_act(bf2f(a.v[e]), bf2f(b.v[e]), act, lim, alpha));
    out[i] = o;
  }
}

// one wave per (row, head): out = x_h / rms(x_h) * w [* silu(gate), or
// sigmoid(gate) with sig]
template <typename T>
__global__ __launch_bounds__(BLOCK) void head_rms_gate_kernel(
    const float* __restrict__ x, const float* __restrict__ w,
    const T* __restrict__ gate, int ldg, T* __restrict__ out, int64_t units,
    int H, int V, float eps, int sig) {
  const int64_t u = (int64_t)blockIdx.x * NW + threadIdx.x / WAVE_SIZE;
  if (u >= units) return;
  const int lane = threadIdx.x & (WAVE_SIZE - 1);
  const float* xr = x + u * V;
  float ss = 0.f;
  for (int c = lane; c < V; c += WAVE_SIZE) ss += xr[c] * xr[c];
  ss = wave_reduce_sum(ss);
  const float rn = 1.0f / sqrtf(ss / (float)V + eps);
  const T* gr = gate ? gate + (u / H) * ldg + (u % H) * V : nullptr;
  for (int c = lane; c < V; c += WAVE_SIZE) {
    float v = xr[c] * rn * w[c];
    if (gate) {
      const float z = ldf<T>(gr, c);
      v *= (sig ? 1.f : z) / (1.f + expf(-z));
    }
    stf<T>(out, u * V + c, v);
  }
}

// the same for V a multiple of 4: LG lanes (a power of two) per (row, head),
// four columns per lane and step
template <typename T>
__global__ __launch_bounds__(BLOCK) void head_rms_gate_vec_kernel(
    const float* __restrict__ x, const float* __restrict__ w,
    const T* __restrict__ gate, int ldg, T* __restrict__ out, int64_t units,
    int H, int V, float eps, int LG, int sig) {
  const int64_t u = ((int64_t)blockIdx.x * BLOCK + threadIdx.x) / LG;
  const bool on = u < units;      // a wave's lanes shuffle together
  const int c0 = (threadIdx.x & (LG - 1)) * 4;
  const float* xr = x + u * V;
  float ss = 0.f;
  if (on)
    for (int c = c0; c < V; c += LG * 4) {
      float v[4];
      ld4(xr + c, v);
#pragma unroll
      for (int e = 0; e < 4; ++e) ss += v[e] * v[e];
    }
  for (int off = LG >> 1; off > 0; off >>= 1)
    ss += __shfl_xor(ss, off, WAVE_SIZE);
  if (!on) return;
  const float rn = 1.0f / sqrtf(ss / (float)V + eps);
  const T* gr = gate ? gate + (u / H) * ldg + (u % H) * V : nullptr;
  for (int c = c0; c < V; c += LG * 4) {
    float v[4], ww[4];
    ld4(xr + c, v);
    ld4(w + c, ww);
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] *= rn * ww[e];
    if (gate) {
      float z[4];
      ld4(gr + c, z);
#pragma unroll
      for (int e = 0; e < 4; ++e)
        v[e] *= (sig ? 1.f : z[e]) / (1.f + expf(-z[e]));
    }
    st4(out + u * V + c, v);
  }
}

template <typename T>
void launch_head_rms(const float* x, const float* w, const T* gate, int ldg,
                     T* out, int64_t units, int H, int V, float eps, int sig,
                     bool vec, hipStream_t stream) {
  if (!vec) {
    hipLaunchKernelGGL(head_rms_gate_kernel<T>,
                       dim3((unsigned)((units + NW - 1) / NW)), dim3(BLOCK), 0,
                       stream, x, w, gate, ldg, out, units, H, V, eps, sig);
    return;
  }
  int LG = 1;
  while (LG < WAVE_SIZE && LG * 4 < V) LG <<= 1;
  hipLaunchKernelGGL(head_rms_gate_vec_kernel<T>,
                     dim3((unsigned)((units * LG + BLOCK - 1) / BLOCK)),
                     dim3(BLOCK), 0, stream, x, w, gate, ldg, out, units, H, V,
                     eps, LG, sig);
}

// out = x / rms(x) * g [* sigmoid(gate)], x fp32 [rows, N]
template <typename T>
__global__ __launch_bounds__(BLOCK) void rms_scale_kernel(
    const float* __restrict__ x, const float* __restrict__ w,
    const T* __restrict__ gate, int ldg, int gate_col, T* __restrict__ out,
    int N, float eps, int one_plus) {
  __shared__ float red[NW];
  const int64_t row = blockIdx.x;
  const float* xr = x + row * N;
  float ss = 0.f;
  for (int c = threadIdx.x; c < N; c += BLOCK) ss += xr[c] * xr[c];
  const float tot = block_reduce_sum<NW>(ss, red);
  const float rn = 1.0f / sqrtf(tot / (float)N + eps);
  for (int c = threadIdx.x; c < N; c += BLOCK) {
    float v = xr[c] * rn * (one_plus ? 1.f + w[c] : w[c]);
    if (gate) {
      const float z = ldf<T>(gate, row * ldg + gate_col + c);
      v *= 1.f / (1.f + expf(-z));
    }
    stf<T>(out, row * N + c, v);
  }
}

template <typename T>
__global__ __launch_bounds__(BLOCK) void gelu_kernel(
    const T* __restrict__ x, T* __restrict__ out, int64_t n, int N,
    int tanh_form, const T* __restrict__ table, int ldt, int table_col,
    const int* __restrict__ tokens) {
  for (int64_t i = (int64_t)blockIdx.x * BLOCK + threadIdx.x; i < n;
       i += (int64_t)gridDim.x * BLOCK) {
    float v = gelu_f(ldf<T>(x, i), tanh_form);
    if (table) {
      const int64_t r = i / N;
      const int c = (int)(i - r * N);
      v *= ldf<T>(table, (int64_t)tokens[r] * ldt + table_col + c);
    }
    stf<T>(out, i, v);
  }
}

// bf16, no gathered factor, n a multiple of 8: 16-byte loads and stores
__global__ __launch_bounds__(BLOCK) void gelu_vec8_kernel(
    const bf16x8* __restrict__ x, bf16x8* __restrict__ out, int64_t n8,
    int tanh_form) {
  for (int64_t i = (int64_t)blockIdx.x * BLOCK + threadIdx.x; i < n8;
       i += (int64_t)gridDim.x * BLOCK) {
    const bf16x8 a = x[i];
    bf16x8 r;
#pragma unroll
    for (int e = 0; e < 8; ++e) r.v[e] = f2bf(gelu_f(bf2f(a.v[e]), tanh_form));
    out[i] = r;
  }
}

// cap 0: the scale alone
__global__ __launch_bounds__(BLOCK) void soft_cap_kernel(float* z, int64_t n,
                                                         float cap,
                                                         float scale) {
  for (int64_t i = (int64_t)blockIdx.x * BLOCK + threadIdx.x; i < n;
       i += (int64_t)gridDim.x * BLOCK) {
    const float v = z[i] * scale;
    z[i] = cap > 0.f ? cap * tanhf(v / cap) : v;
  }
}

int ew_grid(int64_t n) {
  const int64_t b = (n + BLOCK - 1) / BLOCK;
  return (int)(b < 1 ? 1 : (b > 8192 ? 8192 : b));
}

}  // namespace

extern "C" {

void tl_postnorm_add(void* X, const void* y, const void* w, void* h,
                     int64_t rows, int W, float eps, int one_plus, int is_f32,
                     hipStream_t stream) {
  if (rows <= 0) return;
  dim3 grid((unsigned)rows), block(BLOCK);
  if (is_f32)
    hipLaunchKernelGGL(postnorm_add_kernel<float>, grid, block, 0, stream,
                       (float*)X, (const float*)y, (const float*)w,
                       (float*)h, W, eps, one_plus);
  else
    hipLaunchKernelGGL(postnorm_add_kernel<bf16>, grid, block, 0, stream,
                       (float*)X, (const bf16*)y, (const float*)w, (bf16*)h,
                       W, eps, one_plus);
}

// gate: first gate column of row 0 (rows of stride ldg), or null; y, y1, y2
// enter the sum times s0, s1, s2
void tl_add_rms(void* X, const void* y, const void* w, void* h, int64_t rows,
                int W, float eps, float x_scale, const void* gate, int ldg,
                int gate_aligned, float s0, const void* y1, float s1,
                const void* y2, float s2, int is_f32, hipStream_t stream) {
  if (rows <= 0) return;
  const bool vec = W % 4 == 0 && (!gate || gate_aligned);
  if (is_f32)
    launch_add_rms<float>((float*)X, (const float*)y, (const float*)w,
                          (float*)h, rows, W, eps, x_scale,
                          (const float*)gate, ldg,
                          AddMore<float>{(const float*)y1, (const float*)y2,
                                         s0, s1, s2},
                          vec, stream);
  else
    launch_add_rms<bf16>((float*)X, (const bf16*)y, (const float*)w, (bf16*)h,
                         rows, W, eps, x_scale, (const bf16*)gate, ldg,
                         AddMore<bf16>{(const bf16*)y1, (const bf16*)y2, s0,
                                       s1, s2},
                         vec, stream);
}

// p: first gate column of row 0, rows of stride ld
void tl_act_gate(const void* p, int64_t ld, int aligned, void* out,
                 int64_t rows, int N, int act, float lim, float alpha,
                 int is_f32, hipStream_t stream) {
  const int64_t n = rows * N;
  if (n <= 0) return;
  if (!is_f32 && aligned && N % 8 == 0) {
    hipLaunchKernelGGL(act_gate_vec8_kernel, dim3(ew_grid(n / 8)),
                       dim3(BLOCK), 0, stream, (const bf16x8*)p, ld / 8,
                       (bf16x8*)out, n / 8, N / 8, act, lim, alpha);
    return;
  }
  dim3 grid(ew_grid(n)), block(BLOCK);
  if (is_f32)
    hipLaunchKernelGGL(act_gate_kernel<float>, grid, block, 0, stream,
                       (const float*)p, ld, (float*)out, n, N, act, lim, alpha);
  else
    hipLaunchKernelGGL(act_gate_kernel<bf16>, grid, block, 0, stream,
                       (const bf16*)p, ld, (bf16*)out, n, N, act, lim, alpha);
}

void tl_head_rms_gate(const void* x, const void* w, const void* gate, int ldg,
                      int gate_aligned, void* out, int64_t rows, int H, int V,
                      float eps, int sig, int is_f32, hipStream_t stream) {
  const int64_t units = rows * H;
  if (units <= 0) return;
  const bool vec = V % 4 == 0 && (!gate || gate_aligned);
  if (is_f32)
    launch_head_rms<float>((const float*)x, (const float*)w,
                           (const float*)gate, ldg, (float*)out, units, H, V,
                           eps, sig, vec, stream);
  else
    launch_head_rms<bf16>((const float*)x, (const float*)w, (const bf16*)gate,
                          ldg, (bf16*)out, units, H, V, eps, sig, vec,
                          stream);
}

void tl_rms_scale(const void* x, const void* w, const void* gate, int ldg,
                  int gate_col, void* out, int64_t rows, int N, float eps,
                  int one_plus, int is_f32, hipStream_t stream) {
  if (rows <= 0) return;
  dim3 grid((unsigned)rows), block(BLOCK);
  if (is_f32)
    hipLaunchKernelGGL(rms_scale_kernel<float>, grid, block, 0, stream,
                       (const float*)x, (const float*)w, (const float*)gate,
                       ldg, gate_col, (float*)out, N, eps, one_plus);
  else
    hipLaunchKernelGGL(rms_scale_kernel<bf16>, grid, block, 0, stream,
                       (const float*)x, (const float*)w, (const bf16*)gate,
                       ldg, gate_col, (bf16*)out, N, eps, one_plus);
}

void tl_gelu(const void* x, void* out, int64_t n, int N, int tanh_form,
             const void* table, int ldt, int table_col, const void* tokens,
             int is_f32, hipStream_t stream) {
  if (n <= 0) return;
  if (!is_f32 && !table && n % 8 == 0) {
    hipLaunchKernelGGL(gelu_vec8_kernel, dim3(ew_grid(n / 8)), dim3(BLOCK), 0,
                       stream, (const bf16x8*)x, (bf16x8*)out, n / 8,
                       tanh_form);
    return;
  }
  dim3 grid(ew_grid(n)), block(BLOCK);
  if (is_f32)
    hipLaunchKernelGGL(gelu_kernel<float>, grid, block, 0, stream,
                       (const float*)x, (float*)out, n, N, tanh_form,
                       (const float*)table, ldt, table_col,
                       (const int*)tokens);
  else
    hipLaunchKernelGGL(gelu_kernel<bf16>, grid, block, 0, stream,
                       (const bf16*)x, (bf16*)out, n, N, tanh_form,
                       (const bf16*)table, ldt, table_col,
                       (const int*)tokens);
}

void tl_soft_cap(void* z, int64_t n, float cap, float scale,
                 hipStream_t stream) {
  if (n <= 0) return;
  hipLaunchKernelGGL(soft_cap_kernel, dim3(ew_grid(n)), dim3(BLOCK), 0,
                     stream, (float*)z, n, cap, scale);
}

}  // extern "C"
