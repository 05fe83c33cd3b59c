// Shared helpers for the hybrid-mixer kernels (gfx950 / CDNA4).
//
// Every kernel here is templated on the activation storage type: bf16 (held
// as unsigned short, as in the rest of the kernels) or float. All arithmetic
// is fp32; only loads/stores convert.
#pragma once

#include "../ops/common.h"

namespace xllm {
namespace hyb {

template <typename T> struct IO;
template <> struct IO<float> {
  static XLLM_DEV float ld(const float* p) { return *p; }
  static XLLM_DEV void st(float* p, float v) { *p = v; }
  static XLLM_DEV float rnd(float v) { return v; }
};
template <> struct IO<unsigned short> {
  static XLLM_DEV float ld(const unsigned short* p) { return bf16_to_f32(*p); }
  static XLLM_DEV void st(unsigned short* p, float v) { *p = f32_to_bf16(v); }
  static XLLM_DEV float rnd(float v) { return bf16_to_f32(f32_to_bf16(v)); }
};

XLLM_DEV float sigmoidf_(float x) { return 1.0f / (1.0f + __expf(-x)); }
XLLM_DEV float siluf_(float x) { return x / (1.0f + __expf(-x)); }

// two neighbouring values at once (8 B of fp32, 4 B of bf16)
template <typename T> struct Pair;
template <> struct Pair<float> {
  static XLLM_DEV void ld(const float* p, float& a, float& b) {
    const float2 x = *reinterpret_cast<const float2*>(p);
    a = x.x; b = x.y;
  }
  static XLLM_DEV void st(float* p, float a, float b) {
    *reinterpret_cast<float2*>(p) = make_float2(a, b);
  }
};
template <> struct Pair<unsigned short> {
  static XLLM_DEV void ld(const unsigned short* p, float& a, float& b) {
    const unsigned x = *reinterpret_cast<const unsigned*>(p);
    a = bf16_to_f32((unsigned short)(x & 0xffffu));
    b = bf16_to_f32((unsigned short)(x >> 16));
  }
  static XLLM_DEV void st(unsigned short* p, float a, float b) {
    *reinterpret_cast<unsigned*>(p) =
        (unsigned)f32_to_bf16(a) | ((unsigned)f32_to_bf16(b) << 16);
  }
};

// four neighbouring values at once (16 B of fp32, 8 B of bf16)
template <typename T> struct Quad;
template <> struct Quad<float> {
  static XLLM_DEV void ld(const float* p, float v[4]) {
    const float4 x = *reinterpret_cast<const float4*>(p);
    v[0] = x.x; v[1] = x.y; v[2] = x.z; v[3] = x.w;
  }
  static XLLM_DEV void st(float* p, const float v[4]) {
    *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
  }
};
template <> struct Quad<unsigned short> {
  static XLLM_DEV void ld(const unsigned short* p, float v[4]) {
    const ushort4_t x = *reinterpret_cast<const ushort4_t*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = bf16_to_f32(x.x[i]);
  }
  static XLLM_DEV void st(unsigned short* p, const float v[4]) {
    ushort4_t x;
#pragma unroll
    for (int i = 0; i < 4; ++i) x.x[i] = f32_to_bf16(v[i]);
    *reinterpret_cast<ushort4_t*>(p) = x;
  }
};

}  // namespace hyb
}  // namespace xllm
