// Row-wise steps of layers whose mixer and feed-forward read one normed input
// and are added to the residual together.
//
// join_norm: one pass per token over what a layer adds and what reads it next:
//   x[t] <- a * y[row(t)]                                    (entry: no x yet)
//   x[t] <- x[t] + a * y[t] + sum_k wts[t, k] e[rows[t, k]]  (after a layer)
//   h[t]  = x / sqrt(mean(x^2) + eps) * w
// x and all sums fp32; y and e in the activation type; row(t) = ids[t] reads an
// embedding table, t otherwise. e holds the routed experts' outputs, a negative
// row adds nothing. The new x waits in LDS for the norm.
//
// glu_rows: out = act(g) * u * sigmoid(s) for row views, act = SiLU or the
// tanh form of GELU, s one number per row (absent: 1).
#include "hybrid_common.h"

namespace xllm {
namespace hyb {

template <typename T, bool VEC>
__global__ void __launch_bounds__(256) join_norm_kernel(
    float* __restrict__ x, T* __restrict__ h, int fresh,
    const T* __restrict__ y, long y_stride, const long* __restrict__ ids,
    float a, const T* __restrict__ e, const int* __restrict__ rows,
    const float* __restrict__ wts, int top, const float* __restrict__ w,
    float eps, int width) {
  extern __shared__ float row[];          // [width], own entries only
  __shared__ float tmp[16];
  constexpr int N = VEC ? 4 : 1;
  const long t = blockIdx.x;
  float* xr = x + t * width;
  const T* yr = y + (ids != nullptr ? ids[t] : t) * y_stride;
  float ss = 0.f;
  for (int i = threadIdx.x * N; i < width; i += 256 * N) {
    float v[4], z[4];
    if (VEC) Quad<T>::ld(yr + i, v); else v[0] = IO<T>::ld(yr + i);
#pragma unroll
    for (int j = 0; j < N; ++j) v[j] *= a;
    for (int k = 0; k < top; ++k) {
      const int r = rows[t * top + k];
      if (r < 0) continue;
      const float m = wts[t * top + k];
      const T* er = e + (long)r * width + i;
      if (VEC) Quad<T>::ld(er, z); else z[0] = IO<T>::ld(er);
#pragma unroll
      for (int j = 0; j < N; ++j) v[j] += m * z[j];
    }
    if (!fresh) {
      if (VEC) Quad<float>::ld(xr + i, z); else z[0] = xr[i];
#pragma unroll
      for (int j = 0; j < N; ++j) v[j] += z[j];
    }
    if (VEC) { Quad<float>::st(xr + i, v); Quad<float>::st(row + i, v); }
    else { xr[i] = v[0]; row[i] = v[0]; }
#pragma unroll
    for (int j = 0; j < N; ++j) ss += v[j] * v[j];
  }
  ss = block_reduce_sum(ss, tmp);
  const float rs = 1.0f / sqrtf(ss / (float)width + eps);
  T* hr = h + t * width;
  for (int i = threadIdx.x * N; i < width; i += 256 * N) {
    float v[4], z[4];
    if (VEC) { Quad<float>::ld(row + i, v); Quad<float>::ld(w + i, z); }
    else { v[0] = row[i]; z[0] = w[i]; }
#pragma unroll
    for (int j = 0; j < N; ++j) v[j] = v[j] * rs * z[j];
    if (VEC) Quad<T>::st(hr + i, v); else IO<T>::st(hr + i, v[0]);
  }
}

XLLM_DEV float gelu_tanh1_(float z) {
  return 0.5f * z *
         (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

// one workgroup-column of 256 threads walks the quads (or entries) of all rows
template <typename T, bool GELU, bool VEC>
__global__ void __launch_bounds__(256) glu_rows_kernel(
    T* __restrict__ out, long out_stride, const T* __restrict__ g,
    long g_stride, const T* __restrict__ u, long u_stride,
    const T* __restrict__ s, long s_stride, long rows, int F) {
  constexpr int N = VEC ? 4 : 1;
  const int per = F / N;                  // VEC: F % 4 == 0
  const long n = rows * per;
  for (long idx = blockIdx.x * 256L + threadIdx.x; idx < n;
       idx += gridDim.x * 256L) {
    const long r = idx / per;
    const int i = (int)(idx - r * per) * N;
    float a[4], b[4];
    if (VEC) {
      Quad<T>::ld(g + r * g_stride + i, a);
      Quad<T>::ld(u + r * u_stride + i, b);
    } else {
      a[0] = IO<T>::ld(g + r * g_stride + i);
      b[0] = IO<T>::ld(u + r * u_stride + i);
    }
    const float m = s != nullptr ? sigmoidf_(IO<T>::ld(s + r * s_stride)) : 1.f;
#pragma unroll
    for (int j = 0; j < N; ++j)
      a[j] = (GELU ? gelu_tanh1_(a[j]) : siluf_(a[j])) * b[j] * m;
    if (VEC) Quad<T>::st(out + r * out_stride + i, a);
    else IO<T>::st(out + r * out_stride + i, a[0]);
  }
}

template <typename T>
static bool quads_ok(const T* p, long stride) {
  return p == nullptr ||
         (stride % 4 == 0 &&
          reinterpret_cast<uintptr_t>(p) % (4 * sizeof(T)) == 0);
}

template <typename T>
void launch_join_norm(float* x, T* h, int fresh, const T* y, long y_stride,
                      const long* ids, float a, const T* e, const int* rows,
                      const float* wts, int top, const float* w, float eps,
                      long tokens, int width, hipStream_t st) {
  if (tokens == 0) return;
  const bool vec = width % 4 == 0 && quads_ok(y, y_stride) &&
                   quads_ok(e, width) && quads_ok(h, width) &&
                   quads_ok(x, width) && quads_ok(w, width);
  const size_t lds = (size_t)width * sizeof(float);
  if (vec)
    hipLaunchKernelGGL((join_norm_kernel<T, true>), dim3((unsigned)tokens),
                       dim3(256), lds, st, x, h, fresh, y, y_stride, ids, a, e,
                       rows, wts, top, w, eps, width);
  else
    hipLaunchKernelGGL((join_norm_kernel<T, false>), dim3((unsigned)tokens),
                       dim3(256), lds, st, x, h, fresh, y, y_stride, ids, a, e,
                       rows, wts, top, w, eps, width);
}

template <typename T>
void launch_glu_rows(T* out, long out_stride, const T* g, long g_stride,
                     const T* u, long u_stride, const T* s, long s_stride,
                     long rows, int F, int gelu, hipStream_t st) {
  if (rows == 0 || F == 0) return;
  const bool vec = F % 4 == 0 && quads_ok(out, out_stride) &&
                   quads_ok(g, g_stride) && quads_ok(u, u_stride);
  const long n = rows * (vec ? F / 4 : F);
  const int blocks = (int)((n + 255) / 256 < 65535 ? (n + 255) / 256 : 65535);
#define GLU_CALL(G, V)                                                        \
  hipLaunchKernelGGL((glu_rows_kernel<T, G, V>), dim3(blocks), dim3(256), 0,  \
                     st, out, out_stride, g, g_stride, u, u_stride, s,        \
                     s_stride, rows, F)
  if (gelu) { if (vec) GLU_CALL(true, true); else GLU_CALL(true, false); }
  else { if (vec) GLU_CALL(false, true); else GLU_CALL(false, false); }
#undef GLU_CALL
}

#define INST_JL(T)                                                            \
  template void launch_join_norm<T>(float*, T*, int, const T*, long,          \
                                    const long*, float, const T*, const int*, \
                                    const float*, int, const float*, float,   \
                                    long, int, hipStream_t);                  \
  template void launch_glu_rows<T>(T*, long, const T*, long, const T*, long,  \
                                   const T*, long, long, int, int,            \
                                   hipStream_t);
INST_JL(float)
INST_JL(unsigned short)

}  // namespace hyb
}  // namespace xllm
