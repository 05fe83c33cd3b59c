// Retention: linear attention with a fixed decay per head, rotary positions
// on queries and keys, and the gated head norm that follows it.
//
//   S_t = a_h S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t     (S [D, Dv], fp32)
//   y_t = o_t / sqrt(mean(o_t^2) + eps) * silu(g_t)       per head
//
// q and k are turned by the token's position in the half layout (entry i with
// entry i + rot/2) while they are loaded, from a cos/sin table [tokens, rot]
// made once per step (rope_table below), and k is multiplied by k_scale. They
// stay fp32 from there on, for both storage types.
//
// The state lives in a slot pool [slots, H, D, Dv]; a sequence with
// ctx_len == 0 starts from zero whatever its slot held before; slot < 0 runs
// from zero and stores nothing.
//
// Prompt rows run in chunks of 64 tokens of one sequence. Because the decay
// is one number per head, a chunk with the state S before it is
//   O = diag(a^(i+1)) Q S + ((Q K^T) * M) V,   M_ij = a^(i-j) for j <= i
//   S <- a^len S + sum_j a^(len-1-j) k_j v_j^T
// and every product goes to the fp32 matrix pipe (v_mfma_f32_16x16x4_f32,
// true 32-bit products and sums):
//   pass 1  the sum over j of every (chunk, head), all chunks at once
//   scan    chunk after chunk per state element: leaves the state BEFORE each
//           chunk in the chunk's record, the last one in the slot
//   pass 2  the outputs of every (chunk, head), head norm and gate included
// The chunks of a batch are numbered through its sequences without gaps, so
// the scratch holds tokens/64 + sequences records whatever the lengths.
//
// Fragments of the 16x16x4 product (lane l, n = l & 15, g = l >> 4):
//   A[n][g], B[g][n], C[g*4 + r][n].
// The order in which the contraction index is walked is free as long as A and
// B agree. Pass 2 forms S^T = K Q^T, so that a lane's four scores are the
// keys g*4 .. g*4+3 of ONE query, which is what the B operand of
// O^T += V^T P^T wants of that lane: no exchange between lanes. Which value
// column a row of the transposed product stands for is free too: row m of
// product j is column (j / 4) * 64 + m * 4 + j % 4, so a lane fetches the
// operands of four products with one 16 B read and ends up with four
// neighbouring output columns. The key rows of pass 1 are dealt the same way.
#include "hybrid_common.h"

namespace xllm {
namespace hyb {

typedef __attribute__((__vector_size__(4 * sizeof(float)))) float f32x4;

constexpr int RT_C = 64;       // tokens per chunk
constexpr int RT_S = 32;       // tokens staged per LDS fill

// q, k or v rows of a head: stride, columns
template <typename T>
struct RTRows {
  const T* p; long stride; int width;
};
struct RTRot {
  const float* cs; int rot;                       // table [tokens, rot]
};

// Columns c .. c+3 of a row, turned; zeros beyond the width. VEC: widths,
// strides and rot/2 are multiples of four and quads are aligned; addresses are
// clamped instead of branching, so that several of these loads can be in flight
// together.
template <typename T, bool VEC>
XLLM_DEV void rt_load4(const T* row, int c, int width, const float* cs,
                       int rot, float v[4]) {
  const int half = rot >> 1;
  if (VEC) {
    const bool in = c < width;
    Quad<T>::ld(row + (in ? c : 0), v);
    if (rot > 0) {                                // uniform; rot/2 % 4 == 0
      const bool turned = c < rot, first = c < half;
      const int i = turned ? (first ? c : c - half) : 0;
      float y[4], co[4], si[4];
      Quad<T>::ld(row + (first ? i + half : i), y);
      Quad<float>::ld(cs + i, co);
      Quad<float>::ld(cs + half + i, si);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float z = first ? v[j] * co[j] - y[j] * si[j]
                              : v[j] * co[j] + y[j] * si[j];
        v[j] = turned ? z : v[j];
      }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = in ? v[j] : 0.f;
    return;
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int d = c + j;
    float x = 0.f;
    if (d < width) {
      x = IO<T>::ld(row + d);
      if (d < rot) {
        const bool first = d < half;
        const int i = first ? d : d - half;
        const float y = IO<T>::ld(row + (first ? d + half : d - half));
        x = first ? x * cs[i] - y * cs[half + i] : x * cs[i] + y * cs[half + i];
      }
    }
    v[j] = x;
  }
}

// RT_S rows into dst [RT_S][WP + 4], row r times mul (and pw[last - r]); rows
// past `rows` (>= 1) become zeros. B quads per thread are fetched together.
template <typename T, int WP, int B, bool VEC>
XLLM_DEV void rt_stage(float* dst, const RTRows<T>& R, long row0, int rows,
                       const RTRot& rot, float mul, const float* pw, int last) {
  constexpr int N = RT_S * (WP / 4) / 256;        // quads per thread
  static_assert(N % B == 0, "whole batches");
#pragma unroll 1
  for (int b = 0; b < N; b += B) {
    float v[B][4];
#pragma unroll
    for (int i = 0; i < B; ++i) {
      const int idx = threadIdx.x + (b + i) * 256;
      const int r = idx / (WP / 4), c = (idx - r * (WP / 4)) * 4;
      const long t = row0 + min(r, rows - 1);
      rt_load4<T, VEC>(R.p + t * R.stride, c, R.width, rot.cs + t * rot.rot,
                       rot.rot, v[i]);
    }
#pragma unroll
    for (int i = 0; i < B; ++i) {
      const int idx = threadIdx.x + (b + i) * 256;
      const int r = idx / (WP / 4), c = (idx - r * (WP / 4)) * 4;
      const float m = r >= rows ? 0.f : pw != nullptr ? mul * pw[last - r] : mul;
      *reinterpret_cast<float4*>(dst + r * (WP + 4) + c) =
          make_float4(v[i][0] * m, v[i][1] * m, v[i][2] * m, v[i][3] * m);
    }
  }
}

// chunk number b of the batch -> sequence, its chunk, first token, length
XLLM_DEV bool rt_locate(int b, const int* cu_q, int n_seqs, int* s, int* c,
                        int* t0, int* len) {
  int acc = 0;
  for (int i = 0; i < n_seqs; ++i) {
    const int a = cu_q[i], e = cu_q[i + 1];
    const int nc = (e - a + RT_C - 1) / RT_C;
    if (b < acc + nc) {
      *s = i; *c = b - acc;
      *t0 = a + *c * RT_C;
      *len = min(RT_C, e - *t0);
      return true;
    }
    acc += nc;
  }
  return false;
}

// ---- pass 1: what a chunk adds to the state -----------------------------------
// ws [chunks][H][D][Dv]; DP, VP: widths padded to the tile grid; blockIdx.z
// is the block of VP value columns
template <typename T, int DP, int VP, bool VEC>
__global__ void
__launch_bounds__(256, DP == 256 ? 2 : 4) retention_sum_kernel(
    float* __restrict__ ws, RTRows<T> K, RTRows<T> V, RTRot rot, float k_scale,
    const float* __restrict__ decay, const int* __restrict__ cu_q, int n_seqs,
    int heads, int D, int Dv) {
  extern __shared__ float smem[];
  __shared__ float pw[RT_C + 1];
  constexpr int LK = DP + 4, LV = VP + 4;
  constexpr int DT = DP / 64, VT = VP / 16;       // row tiles per wave, columns
  float* ks = smem;                               // [RT_S][LK]
  float* vs = ks + RT_S * LK;                     // [RT_S][LV]
  int s, c, t0, len;
  if (!rt_locate(blockIdx.x, cu_q, n_seqs, &s, &c, &t0, &len)) return;
  const int h = blockIdx.y, v0 = blockIdx.z * VP;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  const int g = lane >> 4, n = lane & 15;
  if (tid <= RT_C) pw[tid] = powf(decay[h], (float)tid);
  __syncthreads();
  K.p += (long)h * D;
  V.p += (long)h * Dv + v0;
  V.width = min(VP, Dv - v0);
  const RTRot none = {nullptr, 0};

  f32x4 acc[DT][VT];
#pragma unroll
  for (int i = 0; i < DT; ++i)
#pragma unroll
    for (int j = 0; j < VT; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int b0 = 0; b0 < len; b0 += RT_S) {
    const int nt = min(RT_S, len - b0);
    if (b0) __syncthreads();
    rt_stage<T, DP, 2, VEC>(ks, K, t0 + b0, nt, rot, k_scale, pw, len - 1 - b0);
    rt_stage<T, VP, 2, VEC>(vs, V, t0 + b0, nt, none, 1.0f, nullptr, 0);
    __syncthreads();
#pragma unroll
    for (int st = 0; st < RT_S / 4; ++st) {
      const float* kr = ks + (st * 4 + g) * LK + w * DT * 16 + n * DT;
      const float* vr = vs + (st * 4 + g) * LV + n * 4;
      float a[DT];
#pragma unroll
      for (int i = 0; i < DT; ++i) a[i] = kr[i];
      float b[VT];
#pragma unroll
      for (int j = 0; j < VT; j += 4) Quad<float>::ld(vr + j * 16, b + j);
#pragma unroll
      for (int j = 0; j < VT; ++j)
#pragma unroll
        for (int i = 0; i < DT; ++i)
          acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(
              a[i], b[j], acc[i][j], 0, 0, 0);
    }
  }
  float* dst = ws + ((long)blockIdx.x * heads + h) * D * (long)Dv + v0;
#pragma unroll
  for (int i = 0; i < DT; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = w * DT * 16 + (g * 4 + r) * DT + i;
      if (d >= D) continue;
#pragma unroll
      for (int j = 0; j < VT; j += 4) {
        const int col = j * 16 + n * 4, left = V.width - col;
        float* p = dst + (long)d * Dv + col;
        const float x[4] = {acc[i][j][r], acc[i][j + 1][r], acc[i][j + 2][r],
                            acc[i][j + 3][r]};
        if (VEC) {
          if (left > 0) Quad<float>::st(p, x);
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (e < left) p[e] = x[e];
        }
      }
    }
}

// ---- scan: one thread per (sequence, state element) -----------------------------
__global__ void retention_scan_kernel(float* __restrict__ ws,
                                      float* __restrict__ state,
                                      const float* __restrict__ decay,
                                      const int* __restrict__ slots,
                                      const int* __restrict__ cu_q,
                                      const int* __restrict__ ctx_lens,
                                      int heads, long per_head) {
  const int s = blockIdx.y;
  const long per_seq = per_head * heads;
  const long e = blockIdx.x * (long)blockDim.x + threadIdx.x;
  if (e >= per_seq) return;
  long base = 0;
  for (int i = 0; i < s; ++i)
    base += (cu_q[i + 1] - cu_q[i] + RT_C - 1) / RT_C;
  const int qlen = cu_q[s + 1] - cu_q[s];
  if (qlen <= 0) return;
  const int full = qlen / RT_C, rest = qlen - full * RT_C;
  const int slot = slots[s];
  const float a = decay[(int)(e / per_head)];
  float S = (slot >= 0 && ctx_lens[s] > 0) ? state[slot * per_seq + e] : 0.f;
  const float a_full = powf(a, (float)RT_C);
  float* w = ws + base * per_seq + e;
  constexpr int U = 8;                    // records in flight
  int c = 0;
  for (; c + U <= full; c += U) {
    float x[U];
#pragma unroll
    for (int i = 0; i < U; ++i) x[i] = w[(c + i) * per_seq];
#pragma unroll
    for (int i = 0; i < U; ++i) {
      w[(c + i) * per_seq] = S;
      S = a_full * S + x[i];
    }
  }
  for (; c < full; ++c) {
    const float x = w[c * per_seq];
    w[c * per_seq] = S;
    S = a_full * S + x;
  }
  if (rest) {
    const float x = w[c * per_seq];
    w[c * per_seq] = S;
    S = powf(a, (float)rest) * S + x;
  }
  if (slot >= 0) state[slot * per_seq + e] = S;
}

// four neighbouring outputs of one head, normed and gated
template <typename T, bool VEC>
XLLM_DEV void rt_store4(T* dst, const T* gate, const f32x4& o, float rs,
                        int n) {
  if (VEC) {
    float gv[4], y[4];
    Quad<T>::ld(gate, gv);
#pragma unroll
    for (int r = 0; r < 4; ++r) y[r] = o[r] * rs * siluf_(gv[r]);
    Quad<T>::st(dst, y);
    return;
  }
#pragma unroll
  for (int r = 0; r < 4; ++r)
    if (r < n) IO<T>::st(dst + r, o[r] * rs * siluf_(IO<T>::ld(gate + r)));
}

// ---- pass 2: the outputs of a chunk ---------------------------------------------
// FUSED (all value columns in one workgroup): y into `out` rows; else the
// plain o into fp32 o_raw [T, H, Dv]. The launch bound keeps the accumulators
// in plain registers (three to four waves per SIMD, no spills).
template <typename T, int DP, int VP, bool FUSED, bool VEC>
__global__ void __launch_bounds__(256, 3) retention_out_kernel(
    T* __restrict__ out, long out_stride, float* __restrict__ o_raw,
    const T* __restrict__ gate, long gate_stride, float eps,
    const float* __restrict__ ws, RTRows<T> Q, RTRows<T> K, RTRows<T> V,
    RTRot rot, float k_scale, const float* __restrict__ decay,
    const int* __restrict__ slots, const int* __restrict__ cu_q,
    const int* __restrict__ ctx_lens, int n_seqs, int heads, int D, int Dv) {
  extern __shared__ float smem[];
  __shared__ float pw[RT_C + 1];
  constexpr int LK = DP + 4, LV = VP + 4;
  constexpr int VT = VP / 16, QT = DP / 16;
  float* ks = smem;                               // [RT_S][LK]
  float* vs = ks + RT_S * LK;                     // [RT_S][LV]
  float* ss = smem;                               // [64][LV], later
  int s, c, t0, len;
  if (!rt_locate(blockIdx.x, cu_q, n_seqs, &s, &c, &t0, &len)) return;
  const int h = blockIdx.y, v0 = blockIdx.z * VP;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  const int g = lane >> 4, n = lane & 15;
  if (tid <= RT_C) pw[tid] = powf(decay[h], (float)tid);
  Q.p += (long)h * D;
  K.p += (long)h * D;
  V.p += (long)h * Dv + v0;
  V.width = min(VP, Dv - v0);
  const RTRot none = {nullptr, 0};
  const int qi = w * 16 + n;                      // this lane's query
  const bool q_ok = qi < len;
  const bool wave_on = w * 16 < len;

  // q[d] at d = i*16 + g*4 + j is the B operand of step (i, j)
  float qv[QT][4];
#pragma unroll
  for (int i = 0; i < QT; ++i) {
    qv[i][0] = qv[i][1] = qv[i][2] = qv[i][3] = 0.f;
    if (q_ok) {
      const long t = t0 + qi;
      rt_load4<T, VEC>(Q.p + t * Q.stride, i * 16 + g * 4, Q.width,
                       rot.cs + t * rot.rot, rot.rot, qv[i]);
    }
  }
  f32x4 acc[VT];
#pragma unroll
  for (int j = 0; j < VT; ++j) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};

  // ---- within the chunk ---------------------------------------------------------
  for (int b0 = 0; b0 < len; b0 += RT_S) {
    __syncthreads();
    rt_stage<T, DP, 2, VEC>(ks, K, t0 + b0, min(RT_S, len - b0), rot, k_scale,
                       nullptr, 0);
    rt_stage<T, VP, VP / 32, VEC>(vs, V, t0 + b0, min(RT_S, len - b0), none, 1.0f,
                             nullptr, 0);
    __syncthreads();
    if (!wave_on) continue;
#pragma unroll
    for (int kt = 0; kt < RT_S / 16; ++kt) {
      const int kb = b0 + kt * 16;                // first key of the tile
      if (kb > w * 16) continue;                  // all later than the queries
      f32x4 p0 = {0.f, 0.f, 0.f, 0.f}, p1 = {0.f, 0.f, 0.f, 0.f};
      const float* kr = ks + (kt * 16 + n) * LK + g * 4;
#pragma unroll
      for (int i = 0; i < QT; ++i) {
        const float4 a = *reinterpret_cast<const float4*>(kr + i * 16);
        p0 = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, qv[i][0], p0, 0, 0, 0);
        p1 = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, qv[i][1], p1, 0, 0, 0);
        p0 = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, qv[i][2], p0, 0, 0, 0);
        p1 = __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, qv[i][3], p1, 0, 0, 0);
      }
      // rows of the score tile: keys kb + g*4 + r, column: query qi
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int back = qi - (kb + g * 4 + r);
        const float p = back >= 0 ? (p0[r] + p1[r]) * pw[back] : 0.f;
        const float* vr = vs + (kt * 16 + g * 4 + r) * LV + n * 4;
        float a[VT];
#pragma unroll
        for (int j = 0; j < VT; j += 4) Quad<float>::ld(vr + j * 16, a + j);
#pragma unroll
        for (int j = 0; j < VT; ++j)
          acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[j], p, acc[j], 0, 0,
                                                        0);
      }
    }
  }
  // ---- through the state before the chunk -----------------------------------------
  if (c > 0 || (slots[s] >= 0 && ctx_lens[s] > 0)) {   // uniform
    const float* S = ws + ((long)blockIdx.x * heads + h) * D * (long)Dv + v0;
    const float fade = pw[min(qi, RT_C - 1) + 1];
#pragma unroll
    for (int sl = 0; sl < DP / 64; ++sl) {
      __syncthreads();
      constexpr int NS = 64 * (VP / 4) / 256;         // quads per thread
      float4 x[NS];
#pragma unroll
      for (int i = 0; i < NS; ++i) {
        const int idx = tid + i * 256;
        const int d = sl * 64 + idx / (VP / 4), cc = idx % (VP / 4) * 4;
        const float* p = S + (long)min(d, D - 1) * Dv;
        if (VEC) {
          x[i] = *reinterpret_cast<const float4*>(p + (cc < V.width ? cc : 0));
        } else {
          const int e = V.width - 1;
          x[i] = make_float4(p[min(cc, e)], p[min(cc + 1, e)],
                             p[min(cc + 2, e)], p[min(cc + 3, e)]);
        }
      }
#pragma unroll
      for (int i = 0; i < NS; ++i) {
        const int idx = tid + i * 256;
        const int d = idx / (VP / 4), cc = idx % (VP / 4) * 4;
        const bool in = sl * 64 + d < D;
        const int left = in ? V.width - cc : 0;       // columns that exist
        *reinterpret_cast<float4*>(ss + d * LV + cc) =
            make_float4(left > 0 ? x[i].x : 0.f, left > 1 ? x[i].y : 0.f,
                        left > 2 ? x[i].z : 0.f, left > 3 ? x[i].w : 0.f);
      }
      __syncthreads();
      if (!wave_on) continue;
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int q4 = 0; q4 < 4; ++q4) {
          const float b = qv[sl * 4 + i][q4] * fade;
          const float* sr = ss + (i * 16 + g * 4 + q4) * LV + n * 4;
          float a[VT];
#pragma unroll
          for (int j = 0; j < VT; j += 4) Quad<float>::ld(sr + j * 16, a + j);
#pragma unroll
          for (int j = 0; j < VT; ++j)
            acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[j], b, acc[j], 0,
                                                          0, 0);
        }
    }
  }
  // acc[j][r] = o[query qi][column v0 + (j/4)*64 + (g*4 + r)*4 + j%4]
  float sq = 0.f;
  if (FUSED) {
#pragma unroll
    for (int j = 0; j < VT; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) sq += acc[j][r] * acc[j][r];
    sq += __shfl_xor(sq, 16, 64);
    sq += __shfl_xor(sq, 32, 64);
  }
  if (!q_ok) return;
  const long t = t0 + qi;
  if (FUSED) {
    const float rs = 1.0f / sqrtf(sq / (float)Dv + eps);
    T* orow = out + t * out_stride + (long)h * Dv;
    const T* grow = gate + t * gate_stride + (long)h * Dv;
#pragma unroll
    for (int j = 0; j < VT; j += 4)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int col = j * 16 + (g * 4 + r) * 4;
        const f32x4 o = {acc[j][r], acc[j + 1][r], acc[j + 2][r],
                         acc[j + 3][r]};
        if (col < Dv)
          rt_store4<T, VEC>(orow + col, grow + col, o, rs, Dv - col);
      }
  } else {
    float* orow = o_raw + (t * heads + h) * (long)Dv + v0;
#pragma unroll
    for (int j = 0; j < VT; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int col = (j & ~3) * 16 + (g * 4 + r) * 4 + (j & 3);
        if (col < V.width) orow[col] = acc[j][r];
      }
  }
}

// ---- decode: one token per sequence -------------------------------------------
// One workgroup per (sequence, head). The step streams the state once in and
// once out: thread (rg, tc) owns VEC neighbouring columns of the rows rg,
// rg + RG, ...; partial outputs of the row groups are summed through LDS,
// where the head norm and the gate follow.
template <typename T, int VEC>
__global__ void __launch_bounds__(256) retention_decode_kernel(
    T* __restrict__ out, long out_stride, const T* __restrict__ gate,
    long gate_stride, float eps, RTRows<T> Q, RTRows<T> K, RTRows<T> V,
    RTRot rot, float k_scale, const float* __restrict__ decay,
    float* __restrict__ state, const int* __restrict__ slots,
    const int* __restrict__ ctx_lens, int heads, int D, int Dv) {
  extern __shared__ float smem[];
  __shared__ float red[4];
  const int Dp = (D + 3) & ~3;      // keeps the regions 16 B aligned
  float* qs = smem;                 // [Dp]
  float* ks = qs + Dp;              // [Dp]
  float* part = ks + Dp;            // [RG][Dv]
  const int s = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int TC = Dv / VEC, RG = 256 / TC;
  const int rg = tid / TC, tc = tid - rg * TC;
  const int half = rot.rot >> 1;
  const float* cs = rot.cs + (long)s * rot.rot;
  const T* qr = Q.p + s * Q.stride + (long)h * D;
  const T* kr = K.p + s * K.stride + (long)h * D;
  for (int i = tid; i < D; i += 256) {
    float a = IO<T>::ld(qr + i), b = IO<T>::ld(kr + i);
    if (i < rot.rot) {
      const bool first = i < half;
      const int f = first ? i : i - half, p = first ? i + half : i - half;
      const float co = cs[f], si = first ? -cs[half + f] : cs[half + f];
      a = a * co + IO<T>::ld(qr + p) * si;
      b = b * co + IO<T>::ld(kr + p) * si;
    }
    qs[i] = a;
    ks[i] = b * k_scale;
  }
  const int slot = slots[s];
  const bool load = slot >= 0 && ctx_lens[s] > 0;
  const float a = decay[h];
  float vv[VEC], o[VEC];
#pragma unroll
  for (int j = 0; j < VEC; ++j) { vv[j] = 0.f; o[j] = 0.f; }
  if (rg < RG) {
    const T* vr = V.p + s * V.stride + (long)h * Dv + tc * VEC;
#pragma unroll
    for (int j = 0; j < VEC; ++j) vv[j] = IO<T>::ld(vr + j);
  }
  __syncthreads();
  if (rg < RG) {
    float* sp = state + (((long)max(slot, 0) * heads + h) * D) * (long)Dv +
                tc * VEC;
#pragma unroll 4
    for (int i = rg; i < D; i += RG) {
      float S[VEC];
#pragma unroll
      for (int j = 0; j < VEC; ++j) S[j] = 0.f;
      if (load) {
        if (VEC == 4) Quad<float>::ld(sp + (long)i * Dv, S);
        else S[0] = sp[(long)i * Dv];
      }
      const float ki = ks[i], qi = qs[i];
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        S[j] = a * S[j] + ki * vv[j];
        o[j] += S[j] * qi;
      }
      if (slot >= 0) {
        if (VEC == 4) Quad<float>::st(sp + (long)i * Dv, S);
        else sp[(long)i * Dv] = S[0];
      }
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) part[rg * Dv + tc * VEC + j] = o[j];
  }
  __syncthreads();
  float sq = 0.f;
  for (int c = tid; c < Dv; c += 256) {
    float y = 0.f;
    for (int r = 0; r < RG; ++r) y += part[r * Dv + c];
    part[c] = y;                    // read and written by this thread alone
    sq += y * y;
  }
  sq = wave_reduce_sum(sq);
  if ((tid & 63) == 0) red[tid >> 6] = sq;
  __syncthreads();
  const float rs =
      1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)Dv + eps);
  T* orow = out + s * out_stride + (long)h * Dv;
  const T* grow = gate + s * gate_stride + (long)h * Dv;
  for (int c = tid; c < Dv; c += 256)
    IO<T>::st(orow + c, part[c] * rs * siluf_(IO<T>::ld(grow + c)));
}

// cos | sin of pos * f_i, angle and sincos in fp64: table [tokens, rot]
__global__ void rope_table_kernel(float* __restrict__ table,
                                  const long* __restrict__ pos,
                                  const double* __restrict__ inv_freq,
                                  int tokens, int half, float mscale) {
  const long idx = blockIdx.x * (long)blockDim.x + threadIdx.x;
  if (idx >= (long)tokens * half) return;
  const long t = idx / half;
  const int i = (int)(idx - t * half);
  double s, c;
  sincos((double)pos[t] * inv_freq[i], &s, &c);
  table[t * 2 * half + i] = (float)(c * mscale);
  table[t * 2 * half + half + i] = (float)(s * mscale);
}

// ---- launchers ------------------------------------------------------------------
void launch_rope_table(float* table, const long* pos, const double* inv_freq,
                       int tokens, int half, float mscale, hipStream_t st) {
  const long n = (long)tokens * half;
  if (n == 0) return;
  hipLaunchKernelGGL(rope_table_kernel, dim3((unsigned)((n + 255) / 256)),
                     dim3(256), 0, st, table, pos, inv_freq, tokens, half,
                     mscale);
}

// records of scratch for a batch of prompt rows
long retention_chunks(long tokens, long n_seqs) {
  return tokens / RT_C + n_seqs;
}
// value columns one workgroup of pass 2 holds: the fused form needs all
int retention_fused_columns() { return 128; }

template <typename T, int DP, int VP, bool VEC>
static void rt_prefill(T* out, long out_stride, float* o_raw, const T* gate,
                       long gate_stride, float eps, float* ws, RTRows<T> Q,
                       RTRows<T> K, RTRows<T> V, RTRot rot, float k_scale,
                       const float* decay, float* state, const int* slots,
                       const int* cu_q, const int* ctx_lens, long tokens,
                       int n_seqs, int heads, int D, int Dv, hipStream_t st) {
  const dim3 grid((unsigned)retention_chunks(tokens, n_seqs), heads,
                  (Dv + VP - 1) / VP);
  const size_t lds = (size_t)RT_S * (DP + 4 + VP + 4) * sizeof(float);
  const size_t lds2 = lds > (size_t)64 * (VP + 4) * sizeof(float)
      ? lds : (size_t)64 * (VP + 4) * sizeof(float);
  hipLaunchKernelGGL((retention_sum_kernel<T, DP, VP, VEC>), grid, dim3(256),
                     lds, st, ws, K, V, rot, k_scale, decay, cu_q, n_seqs,
                     heads, D, Dv);
  const long per_head = (long)D * Dv, per_seq = per_head * heads;
  hipLaunchKernelGGL(retention_scan_kernel,
                     dim3((unsigned)((per_seq + 255) / 256), n_seqs),
                     dim3(256), 0, st, ws, state, decay, slots, cu_q, ctx_lens,
                     heads, per_head);
#define RT_OUT(FUSED)                                                         \
  hipLaunchKernelGGL((retention_out_kernel<T, DP, VP, FUSED, VEC>), grid,     \
                     dim3(256), lds2, st, out, out_stride, o_raw, gate,       \
                     gate_stride, eps, ws, Q, K, V, rot, k_scale, decay,      \
                     slots, cu_q, ctx_lens, n_seqs, heads, D, Dv)
  if (o_raw == nullptr) RT_OUT(true); else RT_OUT(false);
#undef RT_OUT
}

// cu_q == nullptr: decode rows (ws and o_raw unused). o_raw != nullptr: plain
// fp32 outputs there instead of normed and gated ones in `out`.
template <typename T>
void launch_retention(T* out, long out_stride, float* o_raw, const T* gate,
                      long gate_stride, float eps, float* ws, const T* q,
                      const T* k, const T* v, long q_stride, long k_stride,
                      long v_stride, const float* cs, int rot_dims,
                      float k_scale, const float* decay, float* state,
                      const int* slots, const int* cu_q, const int* ctx_lens,
                      long tokens, int n_seqs, int heads, int D, int Dv,
                      hipStream_t st) {
  if (n_seqs == 0 || tokens == 0) return;
  const RTRows<T> Q = {q, q_stride, D}, K = {k, k_stride, D},
                  V = {v, v_stride, Dv};
  const RTRot rot = {cs, rot_dims};
  if (cu_q == nullptr) {
    const int vec = Dv % 4 == 0 ? 4 : 1;
    const int RG = 256 / (Dv / vec);
    const size_t lds =
        (size_t)(2 * ((D + 3) & ~3) + RG * Dv) * sizeof(float);
    if (vec == 4)
      hipLaunchKernelGGL((retention_decode_kernel<T, 4>), dim3(n_seqs, heads),
                         dim3(256), lds, st, out, out_stride, gate,
                         gate_stride, eps, Q, K, V, rot, k_scale, decay, state,
                         slots, ctx_lens, heads, D, Dv);
    else
      hipLaunchKernelGGL((retention_decode_kernel<T, 1>), dim3(n_seqs, heads),
                         dim3(256), lds, st, out, out_stride, gate,
                         gate_stride, eps, Q, K, V, rot, k_scale, decay, state,
                         slots, ctx_lens, heads, D, Dv);
    return;
  }
  auto quads = [](const void* p, long stride, size_t size) {
    return stride % 4 == 0 &&
           reinterpret_cast<uintptr_t>(p) % (4 * size) == 0;
  };
  const bool vec = D % 4 == 0 && Dv % 4 == 0 && rot_dims % 8 == 0 &&
                   quads(cs, rot_dims, 4) && quads(q, q_stride, sizeof(T)) &&
                   quads(k, k_stride, sizeof(T)) &&
                   quads(v, v_stride, sizeof(T)) &&
                   quads(gate, gate_stride, sizeof(T)) &&
                   quads(out, out_stride, sizeof(T));
#define RT_CALL(DP, VP, VEC)                                                  \
  rt_prefill<T, DP, VP, VEC>(out, out_stride, o_raw, gate, gate_stride, eps,  \
                             ws, Q, K, V, rot, k_scale, decay, state, slots,  \
                             cu_q, ctx_lens, tokens, n_seqs, heads, D, Dv, st)
  if (!vec) RT_CALL(256, 128, false);     // odd widths: one size for all
  else if (D <= 64) { if (Dv <= 64) RT_CALL(64, 64, true); else RT_CALL(64, 128, true); }
  else if (D <= 128) { if (Dv <= 64) RT_CALL(128, 64, true); else RT_CALL(128, 128, true); }
  else { if (Dv <= 64) RT_CALL(256, 64, true); else RT_CALL(256, 128, true); }
#undef RT_CALL
}

#define INST_RT(T)                                                            \
  template void launch_retention<T>(                                          \
      T*, long, float*, const T*, long, float, float*, const T*, const T*,    \
      const T*, long, long, long, const float*, int, float, const float*,     \
      float*, const int*, const int*, const int*, long, int, int, int, int,   \
      hipStream_t);
INST_RT(float)
INST_RT(unsigned short)

}  // namespace hyb
}  // namespace xllm
