// Retention prefill on bf16 MFMA 32x32x16, chunks of 128 tokens (head sizes up to 256; other sizes and
// fp32 run retention.hip). Same three steps:
//
//   state   W[c] = V^T K' of chunk c, K' = decayed rotated keys        workgroup: 128 value rows x dim
//   scan    (retention.hip)
//   output  workgroup = chunk, wave = 32 tokens. Everything is held transposed, one token per lane, so
//           the scores' accumulator is the next product's operand, decay^(t+1) is a per-lane scalar
//           and the per-head norm is in-lane plus one xor-32 step:
//             O^T  = S_start Q^T * decay^(t+1)                         (state rows from L2)
//             O^T += V^T (K Q^T o decay^(t-s))                         (64-token tiles in LDS)
//
// Rotated q / k, decayed scores and the state are fp32 values: hi + lo bf16 planes (mma.h).
#include "mix_params.h"
#include "mma.h"

namespace dla {
namespace {

constexpr int kC = 128, kBN = 64, kThreads = 256;
typedef __attribute__((address_space(3))) s16x4 lds_s16x4;

// LDS row strides in elements: rows read 16 B per lane along rows (odd multiple of 16 B), or read
// transposed, 4 rows x 64 B per half wave (odd multiple of 64 B)
__host__ __device__ constexpr int row_stride(int w) { return w + 8; }
__host__ __device__ constexpr int tr_stride(int w) { return w + (w / 32 % 2 ? 0 : 32); }

__device__ __forceinline__ f32x16 mfma32(s16x8 a, s16x8 b, f32x16 c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ s16x4 tr4(const bf16_t* p) { return __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)(p)); }
__device__ __forceinline__ s16x8 cat(s16x4 a, s16x4 b) { return s16x8{a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]}; }

struct Head {
  int b, h, kv0;
  float l2;
};
__device__ __forceinline__ Head head_of(const RetentionParams& p, int h, int b) {
  return Head{b, h, p.kv_start ? p.kv_start[b] : 0, p.decay[p.H + h]};
}

// 8 rotated dimensions of token t0 + t's q or k (zero past len, and for keys in padding)
__device__ __forceinline__ void rotated8(const RetentionParams& p, const Head& hd, int off, int t, int d, int T, bool is_key,
                                         float* v) {
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] = 0.f;
  const int64_t pos = p.base + t - hd.kv0;
  if (t < T && d < p.dim && (pos >= 0 || !is_key)) {
    const int64_t pp = pos < 0 ? 0 : pos;
    const int half = p.rot >> 1;
    load_rotated<bf16_t, 8>(static_cast<const bf16_t*>(p.qkvg) + (static_cast<int64_t>(hd.b) * p.T + t) * p.ld + off, d,
                            p.rot, p.cos_t + pp * half, p.sin_t + pp * half, v);
  }
}
__device__ __forceinline__ bf16x8 value8(const RetentionParams& p, const Head& hd, int off, int t, int v, int T) {
  bf16x8 r = {0, 0, 0, 0, 0, 0, 0, 0};
  if (t < T && v < p.vdim && p.base + t >= hd.kv0)
    r = load_bf16x8(static_cast<const bf16_t*>(p.qkvg) + (static_cast<int64_t>(hd.b) * p.T + t) * p.ld + off + v);
  return r;
}

// grid (nc * ceil(vdim / 128), H, B): wave w = value rows 32 w .. + 31 of the block, all of dim
template <int ND>
__global__ __launch_bounds__(kThreads, ND > 4 ? 1 : 2) void ret_state_mfma_kernel(RetentionParams p) {
  constexpr int DW = 32 * ND, SK = tr_stride(DW), SV = tr_stride(128), CK = DW / 8;
  __shared__ __attribute__((aligned(16))) bf16_t ks[2][kBN * SK];
  __shared__ __attribute__((aligned(16))) bf16_t vs[kBN * SV];
  const Head hd = head_of(p, blockIdx.y, blockIdx.z);
  const int c = blockIdx.x % p.nc, vb = blockIdx.x / p.nc * 128;
  const int t0 = c * kC, len = min(kC, p.T - t0);
  const int Hd = p.H * p.dim;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, c32 = lane & 31, g = lane >> 5;
  f32x16 acc[ND];
#pragma unroll
  for (int n = 0; n < ND; ++n)
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[n][i] = 0.f;
  for (int s0 = 0; s0 < len; s0 += kBN) {
    __syncthreads();
    for (int i = threadIdx.x; i < kBN * CK; i += kThreads) {
      const int t = i / CK, d = (i % CK) * 8;
      float v[8];
      rotated8(p, hd, Hd + hd.h * p.dim, t0 + s0 + t, d, t0 + len, true, v);
      const float f = p.kscale * exp2f(static_cast<float>(len - 1 - s0 - t) * hd.l2);
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = s0 + t < len ? v[e] * f : 0.f;
      s16x8 hi, lo;
      Mma<bf16_t>::split(v, hi, lo);
      store_bf16x8(&ks[0][t * SK + d], __builtin_bit_cast(bf16x8, hi));
      store_bf16x8(&ks[1][t * SK + d], __builtin_bit_cast(bf16x8, lo));
    }
    for (int i = threadIdx.x; i < kBN * 16; i += kThreads) {
      const int t = i >> 4, v = (i & 15) * 8;
      store_bf16x8(vs + t * SV + v, value8(p, hd, 2 * Hd + hd.h * p.vdim, t0 + s0 + t, vb + v, t0 + len));
    }
    __syncthreads();
    // transposed reads: lane's column 16 ((lane >> 4) & 1) + (lane & 15) of a 32-wide tile, rows 8 g .. + 7
    const int tr = (8 * g + ((lane & 15) >> 2)), tc = 16 * ((lane >> 4) & 1) + 4 * (lane & 3);
#pragma unroll
    for (int k = 0; k < kBN; k += 16) {
      const bf16_t* vp = vs + (k + tr) * SV + wave * 32 + tc;
      const s16x8 a = cat(tr4(vp), tr4(vp + 4 * SV));
#pragma unroll
      for (int n = 0; n < ND; ++n) {
        const bf16_t* kp = &ks[0][(k + tr) * SK + 32 * n + tc];
        const bf16_t* kl = &ks[1][(k + tr) * SK + 32 * n + tc];
        acc[n] = mfma32(a, cat(tr4(kp), tr4(kp + 4 * SK)), acc[n]);
        acc[n] = mfma32(a, cat(tr4(kl), tr4(kl + 4 * SK)), acc[n]);
      }
    }
  }
  float* W = p.work + ((static_cast<int64_t>(hd.b) * p.H + hd.h) * p.nc + c) * p.vdim * p.dim;
#pragma unroll
  for (int n = 0; n < ND; ++n)
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int v = vb + wave * 32 + 8 * (i >> 2) + 4 * g + (i & 3), d = 32 * n + c32;
      if (v < p.vdim && d < p.dim) W[static_cast<int64_t>(v) * p.dim + d] = acc[n][i];
    }
}

// grid (nc, H, B). NK: 16-wide steps over dim, NV: 32-wide value tiles
template <int NK, int NV>
__global__ __launch_bounds__(kThreads, NK > 8 ? 1 : 2) void ret_output_mfma_kernel(RetentionParams p) {
  constexpr int SK = row_stride(16 * NK), SV = tr_stride(32 * NV), CK = 2 * NK, CV = 4 * NV;
  __shared__ __attribute__((aligned(16))) bf16_t ks[2][kBN * SK];
  __shared__ __attribute__((aligned(16))) bf16_t vs[kBN * SV];
  const Head hd = head_of(p, blockIdx.y, blockIdx.z);
  const int t0 = blockIdx.x * kC, len = min(kC, p.T - t0);
  const int Hd = p.H * p.dim, Hv = p.H * p.vdim;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, c32 = lane & 31, g = lane >> 5;
  const int tq = wave * 32 + c32;  // this lane's token in the chunk
  s16x8 qh[NK], ql[NK];
#pragma unroll
  for (int s = 0; s < NK; ++s) {
    float v[8];
    rotated8(p, hd, hd.h * p.dim, t0 + tq, 16 * s + 8 * g, t0 + len, false, v);
    Mma<bf16_t>::split(v, qh[s], ql[s]);
  }
  f32x16 o[NV];
#pragma unroll
  for (int t = 0; t < NV; ++t)
#pragma unroll
    for (int i = 0; i < 16; ++i) o[t][i] = 0.f;
  if (!p.fresh || blockIdx.x > 0) {  // (chunk 0 of a fresh sequence starts at zero)
    const float* S = p.work + ((static_cast<int64_t>(hd.b) * p.H + hd.h) * p.nc + blockIdx.x) * p.vdim * p.dim;
    const float f = exp2f(static_cast<float>(tq + 1) * hd.l2);
#pragma unroll
    for (int t = 0; t < NV; ++t) {
      const int v = 32 * t + c32;
      const float* row = S + static_cast<int64_t>(min(v, p.vdim - 1)) * p.dim;
#pragma unroll
      for (int s = 0; s < NK; ++s) {
        const int d = 16 * s + 8 * g;
        float x[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
        if (d < p.dim && v < p.vdim) load_vec<float, 8>(row + d, x);
        s16x8 sh, sl;
        Mma<bf16_t>::split(x, sh, sl);
        o[t] = mfma32(sh, qh[s], o[t]);
        o[t] = mfma32(sl, qh[s], o[t]);
        o[t] = mfma32(sh, ql[s], o[t]);
      }
#pragma unroll
      for (int i = 0; i < 16; ++i) o[t][i] *= f;
    }
  }
  for (int s0 = 0; s0 < len; s0 += kBN) {
    __syncthreads();
    for (int i = threadIdx.x; i < kBN * CK; i += kThreads) {
      const int t = i / CK, d = (i % CK) * 8;
      float v[8];
      rotated8(p, hd, Hd + hd.h * p.dim, t0 + s0 + t, d, t0 + len, true, v);
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] *= p.kscale;
      s16x8 hi, lo;
      Mma<bf16_t>::split(v, hi, lo);
      store_bf16x8(&ks[0][t * SK + d], __builtin_bit_cast(bf16x8, hi));
      store_bf16x8(&ks[1][t * SK + d], __builtin_bit_cast(bf16x8, lo));
    }
    for (int i = threadIdx.x; i < kBN * CV; i += kThreads) {
      const int t = i / CV, v = (i % CV) * 8;
      store_bf16x8(vs + t * SV + v, value8(p, hd, 2 * Hd + hd.h * p.vdim, t0 + s0 + t, v, t0 + len));
    }
    __syncthreads();
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      const int k0 = s0 + 32 * n;  // keys k0 .. k0 + 31 against this wave's tokens 32 wave ..
      if (k0 > wave * 32 + 31) continue;
      f32x16 s;
#pragma unroll
      for (int i = 0; i < 16; ++i) s[i] = 0.f;
#pragma unroll
      for (int k = 0; k < NK; ++k) {
        const s16x8 kh = __builtin_bit_cast(s16x8, load_bf16x8(&ks[0][(32 * n + c32) * SK + 16 * k + 8 * g]));
        const s16x8 kl = __builtin_bit_cast(s16x8, load_bf16x8(&ks[1][(32 * n + c32) * SK + 16 * k + 8 * g]));
        s = mfma32(kh, qh[k], s);
        s = mfma32(kl, qh[k], s);
        s = mfma32(kh, ql[k], s);
      }
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int dt = tq - (k0 + 8 * (i >> 2) + 4 * g + (i & 3));
        s[i] = dt >= 0 ? s[i] * exp2f(static_cast<float>(dt) * hd.l2) : 0.f;
      }
#pragma unroll
      for (int kb = 0; kb < 2; ++kb) {
        float pv[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) pv[e] = s[8 * kb + e];
        s16x8 ph, pl;
        Mma<bf16_t>::split(pv, ph, pl);
        const bf16_t* vp = vs + (32 * n + 16 * kb + 4 * g + ((lane & 15) >> 2)) * SV + 16 * ((lane >> 4) & 1) + 4 * (lane & 3);
#pragma unroll
        for (int t = 0; t < NV; ++t) {
          const s16x8 va = cat(tr4(vp + 32 * t), tr4(vp + 8 * SV + 32 * t));
          o[t] = mfma32(va, ph, o[t]);
          o[t] = mfma32(va, pl, o[t]);
        }
      }
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int t = 0; t < NV; ++t)
#pragma unroll
    for (int i = 0; i < 16; ++i) ss += o[t][i] * o[t][i];  // (rows past vdim are zero)
  ss += __shfl_xor(ss, 32, 64);
  if (tq >= len) return;
  const float rs = rsqrtf(ss / p.vdim + p.eps);
  const int64_t row = static_cast<int64_t>(hd.b) * p.T + t0 + tq;
  const bf16_t* gr = static_cast<const bf16_t*>(p.qkvg) + row * p.ld + 2 * Hd + Hv + hd.h * p.vdim;
  bf16_t* yr = static_cast<bf16_t*>(p.y) + row * Hv + hd.h * p.vdim;
#pragma unroll
  for (int t = 0; t < NV; ++t)
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int v = 32 * t + 8 * u + 4 * g;
      if (v >= p.vdim) continue;
      const bf16x4 gv = *reinterpret_cast<const bf16x4*>(gr + v);
      float y[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float z = bf2f(gv[e]);
        y[e] = o[t][4 * u + e] * rs * (z / (1.f + __expf(-z)));
      }
      typedef uint32_t u32x2 __attribute__((ext_vector_type(2)));
      *reinterpret_cast<u32x2*>(yr + v) = u32x2{pack2bf(y[0], y[1]), pack2bf(y[2], y[3])};
    }
}

}  // namespace

bool retention_mfma_ok(const RetentionParams& p) {
  return p.dim % 8 == 0 && p.vdim % 8 == 0 && p.rot % 16 == 0 && p.ld % 8 == 0 && p.dim <= 256 && p.vdim <= 256 &&
         reinterpret_cast<uintptr_t>(p.qkvg) % 16 == 0 && reinterpret_cast<uintptr_t>(p.y) % 16 == 0;
}

void launch_retention_state_mfma(const RetentionParams& p, hipStream_t st) {
  const dim3 g(p.nc * ((p.vdim + 127) / 128), p.H, p.B);
  if (p.dim <= 64) ret_state_mfma_kernel<2><<<g, kThreads, 0, st>>>(p);
  else if (p.dim <= 128) ret_state_mfma_kernel<4><<<g, kThreads, 0, st>>>(p);
  else ret_state_mfma_kernel<8><<<g, kThreads, 0, st>>>(p);
}

void launch_retention_output_mfma(const RetentionParams& p, hipStream_t st) {
  const dim3 g(p.nc, p.H, p.B);
  if (p.dim <= 64 && p.vdim <= 64) ret_output_mfma_kernel<4, 2><<<g, kThreads, 0, st>>>(p);
  else if (p.dim <= 128 && p.vdim <= 128) ret_output_mfma_kernel<8, 4><<<g, kThreads, 0, st>>>(p);
  else ret_output_mfma_kernel<16, 8><<<g, kThreads, 0, st>>>(p);
}

}  // namespace dla
