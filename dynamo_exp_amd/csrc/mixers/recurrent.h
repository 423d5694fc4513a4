// Shared by the kernels with per-sequence state: element access, activations,
// sums over lane groups by DPP exchanges, 16-byte vector access, dispatch over
// the activation element.
#pragma once
#include "../kernels/common.h"

namespace {

constexpr int kRows = 16;  // state rows per thread
constexpr int kTok = 8;    // tokens per staged block

template <typename T> __device__ __forceinline__ float ldf(const T* p, int64_t i);
template <> __device__ __forceinline__ float ldf<bf16_t>(const bf16_t* p, int64_t i) { return bf16_to_f32(p[i]); }
template <> __device__ __forceinline__ float ldf<float>(const float* p, int64_t i) { return p[i]; }
template <typename T> __device__ __forceinline__ void stf(T* p, int64_t i, float v);
template <> __device__ __forceinline__ void stf<bf16_t>(bf16_t* p, int64_t i, float v) { p[i] = f32_to_bf16(v); }
template <> __device__ __forceinline__ void stf<float>(float* p, int64_t i, float v) { p[i] = v; }

__device__ __forceinline__ float sigmoidf_(float z) { return 1.f / (1.f + expf(-z)); }

// the same from the hardware's exp2 and reciprocal (relative error a few 1e-7): per-element gates of wide rows
__device__ __forceinline__ float fast_sigmoid(float z) {
  return __builtin_amdgcn_rcpf(1.f + fast_exp2(z * -1.4426950408889634f));
}

template <int CTRL> __device__ __forceinline__ float dpp_f(float v) {
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xf, 0xf, false));
}
// sum over the R lanes of an aligned lane group (R <= 16), the result in every lane of the group:
// neighbours within a quad, the other pair of the quad, the other quad of a half row (half-row
// mirror: the quads already hold one value each), the other half of a row of 16 (row mirror)
template <int R> __device__ __forceinline__ float group_sum(float v) {
  if constexpr (R >= 2) v += dpp_f<0xB1>(v);
  if constexpr (R >= 4) v += dpp_f<0x4E>(v);
  if constexpr (R >= 8) v += dpp_f<0x141>(v);
  if constexpr (R >= 16) v += dpp_f<0x140>(v);
  return v;
}

template <typename T, int V> struct VecIO;
template <> struct VecIO<bf16_t, 8> {
  __device__ static __forceinline__ void ld(const bf16_t* p, float* o) {
    const u16x8 a = *reinterpret_cast<const u16x8*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) o[2 * i] = bf16lo(a.w[i]), o[2 * i + 1] = bf16hi(a.w[i]);
  }
  __device__ static __forceinline__ void st(bf16_t* p, const float* v) {
    u16x8 a;
#pragma unroll
    for (int i = 0; i < 4; ++i) a.w[i] = pack_bf16x2(v[2 * i], v[2 * i + 1]);
    *reinterpret_cast<u16x8*>(p) = a;
  }
};
// 16 raw bytes as floats
typedef uint32_t raw_u32x4 __attribute__((ext_vector_type(4)));
template <typename T> __device__ __forceinline__ void chunk_to_f32(const raw_u32x4& c, float* o);
template <> __device__ __forceinline__ void chunk_to_f32<bf16_t>(const raw_u32x4& c, float* o) {
#pragma unroll
  for (int i = 0; i < 4; ++i) o[2 * i] = bf16lo(c[i]), o[2 * i + 1] = bf16hi(c[i]);
}
template <> __device__ __forceinline__ void chunk_to_f32<float>(const raw_u32x4& c, float* o) {
#pragma unroll
  for (int i = 0; i < 4; ++i) o[i] = __uint_as_float(c[i]);
}
template <> struct VecIO<float, 4> {
  __device__ static __forceinline__ void ld(const float* p, float* o) {
    const f32x4 a = *reinterpret_cast<const f32x4*>(p);
    o[0] = a[0], o[1] = a[1], o[2] = a[2], o[3] = a[3];
  }
  __device__ static __forceinline__ void st(float* p, const float* v) {
    *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
  }
};

}  // namespace

#define DISPATCH_T(f32, ...)          \
  if (f32) {                          \
    using T = float;                  \
    __VA_ARGS__;                      \
  } else {                            \
    using T = bf16_t;                 \
    __VA_ARGS__;                      \
  }
