// A layer's result, the weighted sum over the depth, and the next layer's two
// normed inputs, in one pass over a token's row; two row-wise activations.
//
// depth_mix_norm, one workgroup per token:
//   r     = x_in + m_scale (m1' + m2') + f           -> hist[level]
//   x_out = sum_{j <= level} dwa[j] hist[j]
//   h1, h2 = x_out / rms(x_out) * g1 | g2            (one number each)
// with m' = m / rms(m) * w where a weight is given (one per column or a single
// number) and m' = m otherwise. rms(z) = sqrt(mean(z^2) + eps). m1, m2 are in
// the activation type, f in that type or fp32; the residual, the results
// hist [levels, T, W] and all sums are fp32. The new row waits in LDS between
// its sum of squares and the normed writes, so every operand is read once.
//
// clamped_glu: g = min(a, limit), u = clamp(b, +-limit) for the halves a | b
// of a row: out = g sigmoid(alpha g) (u + shift).
//
// gelu_scaled: out[r] = gelu(s_r x[r]), exact (erf). s_r from a vector, or for
// rows in the order (expert, token) the weight with which the token chose that
// expert; rows no token chose become zero and are not read.
#include "hybrid_common.h"

namespace xllm {
namespace hyb {

template <typename T, int V>
XLLM_DEV void ldv(const T* p, float v[V]) {
  if (V == 4) Quad<T>::ld(p, v);
  else v[0] = IO<T>::ld(p);
}
template <typename T, int V>
XLLM_DEV void stv(T* p, const float v[V]) {
  if (V == 4) Quad<T>::st(p, v);
  else IO<T>::st(p, v[0]);
}

struct DMArgs {
  const float* x_in; float* x_out; float* hist;
  const float* w1; const float* w2; int w1_n, w2_n;   // weights: 1 or W
  const float* dwa; const float* g1; const float* g2;
  float m_scale, eps;
  int level, W;
  long level_stride;
};

template <typename T, int V>
XLLM_DEV float dm_sum_sq(const T* row, int W) {
  float ss = 0.f;
  for (int c = threadIdx.x * V; c < W; c += 256 * V) {
    float v[V];
    ldv<T, V>(row + c, v);
#pragma unroll
    for (int i = 0; i < V; ++i) ss += v[i] * v[i];
  }
  return ss;
}

// V = 4: four columns per access (W a multiple of 4), V = 1: any width
template <typename T, typename TF, int V>
__global__ void __launch_bounds__(256) depth_mix_norm_kernel(
    T* __restrict__ h1, T* __restrict__ h2, DMArgs A,
    const T* __restrict__ m1, const T* __restrict__ m2,
    const TF* __restrict__ f) {
  extern __shared__ float u[];             // [W] the new residual row
  __shared__ float tmp[16];
  const int W = A.W, tid = threadIdx.x;
  const long row = (long)blockIdx.x * W;
  float r1 = 1.f, r2 = 1.f;
  if (A.w1) {
    r1 = block_reduce_sum(dm_sum_sq<T, V>(m1 + row, W), tmp);
    r1 = 1.0f / sqrtf(r1 / (float)W + A.eps);
    __syncthreads();
  }
  if (m2 != nullptr && A.w2) {
    r2 = block_reduce_sum(dm_sum_sq<T, V>(m2 + row, W), tmp);
    r2 = 1.0f / sqrtf(r2 / (float)W + A.eps);
    __syncthreads();
  }
  float ss = 0.f;
  for (int c = tid * V; c < W; c += 256 * V) {
    float r[V], t[V];
    ldv<T, V>(m1 + row + c, r);
    if (A.w1) {
#pragma unroll
      for (int i = 0; i < V; ++i)
        r[i] *= r1 * A.w1[A.w1_n == 1 ? 0 : c + i];
    }
    if (m2 != nullptr) {
      ldv<T, V>(m2 + row + c, t);
#pragma unroll
      for (int i = 0; i < V; ++i)
        r[i] += t[i] * (A.w2 ? r2 * A.w2[A.w2_n == 1 ? 0 : c + i] : 1.f);
    }
#pragma unroll
    for (int i = 0; i < V; ++i) r[i] *= A.m_scale;
    if (f != nullptr) {
      ldv<TF, V>(f + row + c, t);
#pragma unroll
      for (int i = 0; i < V; ++i) r[i] += t[i];
    }
    if (A.x_in != nullptr) {
      ldv<float, V>(A.x_in + row + c, t);
#pragma unroll
      for (int i = 0; i < V; ++i) r[i] += t[i];
    }
    float* hp = A.hist + row + c;
    stv<float, V>(hp + A.level * A.level_stride, r);
    if (A.dwa != nullptr) {
      const float wl = A.dwa[A.level];
#pragma unroll
      for (int i = 0; i < V; ++i) r[i] *= wl;
#pragma unroll 4
      for (int j = 0; j < A.level; ++j) {
        float o[V];
        ldv<float, V>(hp + j * A.level_stride, o);
        const float wj = A.dwa[j];
#pragma unroll
        for (int i = 0; i < V; ++i) r[i] += wj * o[i];
      }
    }
    if (A.x_out != nullptr) stv<float, V>(A.x_out + row + c, r);
#pragma unroll
    for (int i = 0; i < V; ++i) { u[c + i] = r[i]; ss += r[i] * r[i]; }
  }
  ss = block_reduce_sum(ss, tmp);
  const float rs = 1.0f / sqrtf(ss / (float)W + A.eps);
  const float s1 = rs * A.g1[0];
  const float s2 = h2 != nullptr ? rs * A.g2[0] : 0.f;
  for (int c = tid * V; c < W; c += 256 * V) {   // a thread's own entries
    float a[V], b[V];
#pragma unroll
    for (int i = 0; i < V; ++i) { a[i] = u[c + i] * s1; b[i] = u[c + i] * s2; }
    stv<T, V>(h1 + row + c, a);
    if (h2 != nullptr) stv<T, V>(h2 + row + c, b);
  }
}

template <typename T, int V>
__global__ void __launch_bounds__(256) clamped_glu_kernel(
    T* __restrict__ out, const T* __restrict__ x, long rows, int F,
    float limit, float alpha, float shift) {
  const int per = F / V;
  const long n = rows * (long)per;
  for (long idx = blockIdx.x * 256L + threadIdx.x; idx < n;
       idx += gridDim.x * 256L) {
    const long r = idx / per;
    const int c = (int)(idx - r * per) * V;
    float a[V], b[V];
    ldv<T, V>(x + r * 2 * F + c, a);
    ldv<T, V>(x + r * 2 * F + F + c, b);
#pragma unroll
    for (int i = 0; i < V; ++i) {
      const float g = fminf(a[i], limit);
      const float y = fminf(fmaxf(b[i], -limit), limit);
      a[i] = g * sigmoidf_(alpha * g) * (y + shift);
    }
    stv<T, V>(out + r * F + c, a);
  }
}

template <typename T, int V>
__global__ void __launch_bounds__(256) gelu_scaled_kernel(
    T* __restrict__ out, const T* __restrict__ x, long rows, int F,
    const float* __restrict__ scale, const int* __restrict__ ids,
    const float* __restrict__ wts, int tokens, int top) {
  const int per = F / V;
  const long n = rows * (long)per;
  for (long idx = blockIdx.x * 256L + threadIdx.x; idx < n;
       idx += gridDim.x * 256L) {
    const long r = idx / per;
    const int c = (int)(idx - r * per) * V;
    float s = scale != nullptr ? scale[r] : 1.f;
    bool used = true;
    if (ids != nullptr) {
      const int e = (int)(r / tokens), t = (int)(r - (long)e * tokens);
      used = false;
      for (int k = 0; k < top; ++k)
        if (ids[(long)t * top + k] == e) { s = wts[(long)t * top + k]; used = true; }
    }
    float a[V];
#pragma unroll
    for (int i = 0; i < V; ++i) a[i] = 0.f;
    if (used) {
      ldv<T, V>(x + r * F + c, a);
#pragma unroll
      for (int i = 0; i < V; ++i) {
        const float z = s * a[i];
        a[i] = 0.5f * z * (1.0f + erff(z * 0.70710678118654752f));
      }
    }
    stv<T, V>(out + r * F + c, a);
  }
}

static inline int blocks_of(long n) {
  const long b = (n + 255) / 256;
  return (int)(b < 65535 ? b : 65535);
}

template <typename T, typename TF>
void launch_depth_mix_norm(T* h1, T* h2, float* x_out, const float* x_in,
                           float* hist, long level_stride, int level,
                           const T* m1, const float* w1, int w1_n,
                           const T* m2, const float* w2, int w2_n,
                           float m_scale, const TF* f, const float* dwa,
                           const float* g1, const float* g2, float eps,
                           int tokens, int W, hipStream_t st) {
  if (tokens == 0) return;
  const DMArgs A{x_in, x_out, hist, w1, w2, w1_n, w2_n, dwa, g1, g2,
                 m_scale, eps, level, W, level_stride};
  const size_t lds = (size_t)W * sizeof(float);
  if (W % 4 == 0)
    hipLaunchKernelGGL((depth_mix_norm_kernel<T, TF, 4>), dim3(tokens),
                       dim3(256), lds, st, h1, h2, A, m1, m2, f);
  else
    hipLaunchKernelGGL((depth_mix_norm_kernel<T, TF, 1>), dim3(tokens),
                       dim3(256), lds, st, h1, h2, A, m1, m2, f);
}

template <typename T>
void launch_clamped_glu(T* out, const T* x, long rows, int F, float limit,
                        float alpha, float shift, hipStream_t st) {
  if (rows * F == 0) return;
  if (F % 4 == 0)
    hipLaunchKernelGGL((clamped_glu_kernel<T, 4>), dim3(blocks_of(rows * F / 4)),
                       dim3(256), 0, st, out, x, rows, F, limit, alpha, shift);
  else
    hipLaunchKernelGGL((clamped_glu_kernel<T, 1>), dim3(blocks_of(rows * F)),
                       dim3(256), 0, st, out, x, rows, F, limit, alpha, shift);
}

template <typename T>
void launch_gelu_scaled(T* out, const T* x, long rows, int F,
                        const float* scale, const int* ids, const float* wts,
                        int tokens, int top, hipStream_t st) {
  if (rows * F == 0) return;
  if (F % 4 == 0)
    hipLaunchKernelGGL((gelu_scaled_kernel<T, 4>), dim3(blocks_of(rows * F / 4)),
                       dim3(256), 0, st, out, x, rows, F, scale, ids, wts,
                       tokens, top);
  else
    hipLaunchKernelGGL((gelu_scaled_kernel<T, 1>), dim3(blocks_of(rows * F)),
                       dim3(256), 0, st, out, x, rows, F, scale, ids, wts,
                       tokens, top);
}

#define INST_DM(T, TF)                                                        \
  template void launch_depth_mix_norm<T, TF>(                                 \
      T*, T*, float*, const float*, float*, long, int, const T*,              \
      const float*, int, const T*, const float*, int, float, const TF*,       \
      const float*, const float*, const float*, float, int, int, hipStream_t);
INST_DM(float, float)
INST_DM(unsigned short, float)
INST_DM(unsigned short, unsigned short)

#define INST_ACT(T)                                                           \
  template void launch_clamped_glu<T>(T*, const T*, long, int, float, float,  \
                                      float, hipStream_t);                    \
  template void launch_gelu_scaled<T>(T*, const T*, long, int, const float*,  \
                                      const int*, const float*, int, int,     \
                                      hipStream_t);
INST_ACT(float)
INST_ACT(unsigned short)

}  // namespace hyb
}  // namespace xllm
