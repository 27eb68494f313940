// MFMA tiles for element types bf16 and fp32, shared by the mixer kernels (latent attention,
// retention). One 16 x 16 output tile per wave: C[m = 4 (lane / 16) + i][n = lane % 16].
//
//   bf16  v_mfma_f32_16x16x32_bf16, k-step 32, lane holds 8 consecutive k
//   fp32  4 x v_mfma_f32_16x16x4_f32, k-step 16, lane holds 4 consecutive k (k slot j of lane group
//         g is k = 4g + j on both operands, so the order of the sum is permuted, nothing else)
//
// Values that have to stay fp32 while the kernel runs on bf16 MFMAs (softmax weights, decayed
// scores, rotated keys on their way into a state, the state itself) travel as two bf16 planes,
// hi = bf16(x) and lo = bf16(x - hi): products against both planes keep 16 mantissa bits. The fp32
// kernels have one plane.
#pragma once
#include "../common.h"

namespace dla {

template <typename T>
struct Mma;

template <>
struct Mma<bf16_t> {
  using Frag = s16x8;
  static constexpr int KS = 32;  // k per step
  static constexpr int KV = 8;   // k per lane
  static constexpr int PL = 2;   // planes of an fp32-valued operand
  static __device__ __forceinline__ Frag zero() { return Frag{0, 0, 0, 0, 0, 0, 0, 0}; }
  static __device__ __forceinline__ Frag row(const bf16_t* p) { return __builtin_bit_cast(s16x8, load_bf16x8(p)); }
  static __device__ __forceinline__ Frag col(const bf16_t* p, int ld) {
    Frag f;
#pragma unroll
    for (int j = 0; j < 8; ++j) f[j] = static_cast<short>(p[j * ld]);
    return f;
  }
  static __device__ __forceinline__ void set(Frag& f, int e, bf16_t v) { f[e] = static_cast<short>(v); }
  static __device__ __forceinline__ f32x4 mma(Frag a, Frag b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
  }
  // x[8] -> hi and lo fragments
  static __device__ __forceinline__ void split(const float* x, Frag& hi, Frag& lo) {
    float r[8];
    const bf16x8 h = pack_bf16x8(x);
#pragma unroll
    for (int j = 0; j < 8; ++j) r[j] = x[j] - bf2f(h[j]);
    hi = __builtin_bit_cast(s16x8, h);
    lo = __builtin_bit_cast(s16x8, pack_bf16x8(r));
  }
};

template <>
struct Mma<float> {
  using Frag = f32x4;
  static constexpr int KS = 16;
  static constexpr int KV = 4;
  static constexpr int PL = 1;
  static __device__ __forceinline__ Frag zero() { return Frag{0.f, 0.f, 0.f, 0.f}; }
  static __device__ __forceinline__ Frag row(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
  static __device__ __forceinline__ Frag col(const float* p, int ld) { return Frag{p[0], p[ld], p[2 * ld], p[3 * ld]}; }
  static __device__ __forceinline__ void set(Frag& f, int e, float v) { f[e] = v; }
  static __device__ __forceinline__ f32x4 mma(Frag a, Frag b, f32x4 c) {
#pragma unroll
    for (int j = 0; j < 4; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[j], b[j], c, 0, 0, 0);
    return c;
  }
  static __device__ __forceinline__ void split(const float* x, Frag& hi, Frag& lo) {
    hi = Frag{x[0], x[1], x[2], x[3]};
    lo = zero();
  }
};

template <typename T>
__device__ __forceinline__ float to_f(T v);
template <>
__device__ __forceinline__ float to_f<bf16_t>(bf16_t v) { return bf2f(v); }
template <>
__device__ __forceinline__ float to_f<float>(float v) { return v; }

template <typename T>
__device__ __forceinline__ T from_f(float v);
template <>
__device__ __forceinline__ bf16_t from_f<bf16_t>(float v) { return f2bf(v); }
template <>
__device__ __forceinline__ float from_f<float>(float v) { return v; }

// store an fp32 value as its planes (plane stride in elements)
template <typename T>
__device__ __forceinline__ void put_planes(T* p, int plane, float v);
template <>
__device__ __forceinline__ void put_planes<bf16_t>(bf16_t* p, int plane, float v) {
  const bf16_t h = f2bf(v);
  p[0] = h;
  p[plane] = f2bf(v - bf2f(h));
}
template <>
__device__ __forceinline__ void put_planes<float>(float* p, int, float v) { p[0] = v; }

// VEC consecutive elements -> fp32 (8- or 16-byte loads; the caller checks alignment)
template <typename T, int VEC>
__device__ __forceinline__ void load_vec(const T* p, float* o) {
  if constexpr (VEC == 8 && sizeof(T) == 2) {
    const bf16x8 v = load_bf16x8(reinterpret_cast<const bf16_t*>(p));
#pragma unroll
    for (int j = 0; j < 8; ++j) o[j] = bf2f(v[j]);
  } else if constexpr (VEC == 4 && sizeof(T) == 2) {
    const bf16x4 v = *reinterpret_cast<const bf16x4*>(p);
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] = bf2f(v[j]);
  } else if constexpr (VEC % 4 == 0 && sizeof(T) == 4) {
#pragma unroll
    for (int j = 0; j < VEC; j += 4) {
      const f32x4 v = *reinterpret_cast<const f32x4*>(p + j);
      o[j] = v[0]; o[j + 1] = v[1]; o[j + 2] = v[2]; o[j + 3] = v[3];
    }
  } else {
#pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] = to_f<T>(p[j]);
  }
}

template <typename T, int VEC>
__device__ __forceinline__ void store_vec(T* p, const float* v) {
  if constexpr (VEC == 8 && sizeof(T) == 2) {
    store_bf16x8(reinterpret_cast<bf16_t*>(p), pack_bf16x8(v));
  } else if constexpr (VEC == 4 && sizeof(T) == 2) {
    typedef uint32_t u32x2 __attribute__((ext_vector_type(2)));
    *reinterpret_cast<u32x2*>(p) = u32x2{pack2bf(v[0], v[1]), pack2bf(v[2], v[3])};
  } else if constexpr (VEC % 4 == 0 && sizeof(T) == 4) {
#pragma unroll
    for (int j = 0; j < VEC; j += 4) *reinterpret_cast<f32x4*>(p + j) = f32x4{v[j], v[j + 1], v[j + 2], v[j + 3]};
  } else {
#pragma unroll
    for (int j = 0; j < VEC; ++j) p[j] = from_f<T>(v[j]);
  }
}

// Dimensions i0 .. i0 + VEC - 1 of a head vector after rotary positions on its first `rot` dimensions
// (dimension i < rot / 2 pairs with i + rot / 2); cs / sn: the position's table rows [rot / 2].
// VEC divides rot / 2 (or rot == 0), so a vector never straddles a pair boundary.
template <typename T, int VEC>
__device__ __forceinline__ void load_rotated(const T* p, int i0, int rot, const float* cs, const float* sn, float* o) {
  load_vec<T, VEC>(p + i0, o);
  if (i0 >= rot) return;
  const int half = rot >> 1;
  float w[VEC];
  if (i0 < half) {
    load_vec<T, VEC>(p + i0 + half, w);
#pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] = o[j] * cs[i0 + j] - w[j] * sn[i0 + j];
  } else {
    load_vec<T, VEC>(p + i0 - half, w);
#pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] = o[j] * cs[i0 - half + j] + w[j] * sn[i0 - half + j];
  }
}

// 0.5 z (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3))), the tanh as 1 - 2 / (1 + e^(2u))
__device__ __forceinline__ float gelu_tanh(float z) {
  const float u = 0.7978845608028654f * (z + 0.044715f * z * z * z);
  return z * (1.f - 1.f / (1.f + __expf(2.f * u)));
}

__host__ __device__ constexpr int round_up(int x, int m) { return (x + m - 1) / m * m; }

}  // namespace dla
