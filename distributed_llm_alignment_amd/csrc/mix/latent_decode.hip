// Latent-attention decode on the latent cache, bf16: kv_rank <= 512, kv_rank + rot <= 576 (other sizes and
// fp32: latent.hip).
//
// Workgroup = (key split, group of 16 heads, sequence), 4 waves. A tile of 64 cache rows is read once
// for all heads, straight into LDS (LDS-DMA, the whole tile in flight, no registers), kept as one
// XOR-swizzled row image and used twice: as keys along its rows (wave w: 16 of the
// 64 keys against the 16 heads) and as values along its columns by transposed reads (wave w: every
// fourth 16-column tile of the latent). Softmax weights are fp32, in the product as hi + lo planes.
#include "mix_params.h"
#include "mma.h"

namespace dla {
namespace {

constexpr float kLog2e = 1.4426950408889634f;
constexpr int kBN = 64, kSS = kBN + 4, kSP = 2 * kSS;  // score row: 272 bytes (an odd multiple of 16)
typedef __attribute__((address_space(3))) s16x4 lds_s16x4;
__device__ __forceinline__ s16x4 tr4(const bf16_t* p) { return __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)(p)); }

// Position of 16-byte chunk c of row n in the image (rows of NV = 8 (mod 16) chunks). The XOR inside
// aligned groups of 8 chunks spreads both a column of 16 rows (score fragments) and 4 rows x 32 bytes
// (transposed reads) over all banks.
__device__ __forceinline__ int img_f(int n) { return ((n >> 1) & 1) << 1 | ((n >> 2) & 1) << 2 | ((n >> 3) & 1); }
template <int NV>
__device__ __forceinline__ int img(int n, int c) { return (n * NV + (c ^ img_f(n))) * 8; }

// NK: 32-wide steps over kv_rank + rot, NT: 16-column latent tiles per wave
template <int NK, int NT>
__global__ __launch_bounds__(256, 2) void latent_decode_mfma_kernel(LatentParams p) {
  constexpr int NV = 4 * NK;  // 16-byte chunks per row
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  bf16_t* ls = reinterpret_cast<bf16_t*>(smem);
  // one row per head: 64 fp32 scores, overwritten in place by their weights' planes (64 hi, 64 lo)
  bf16_t* ps = ls + kBN * 8 * NV;
  float* ss = reinterpret_cast<float*>(ps);
  float* al = ss + 16 * kSS;
  const int split = blockIdx.x, h0 = blockIdx.y * 16, b = blockIdx.z;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane & 15, g = lane >> 4;
  const int lq = p.R + p.rot, nh = min(16, p.H - h0);
  const int newest = static_cast<int>(min(p.slot[0], static_cast<int64_t>(p.tcap - 1)));
  int lo = p.kv_start ? p.kv_start[b] : 0;
  if (p.window) lo = max(lo, newest - p.window + 1);
  int per = (newest - lo + p.ns) / p.ns;
  per = (per + kBN - 1) / kBN * kBN;
  const int k0 = lo + split * per, k1 = min(k0 + per, newest + 1);
  const bf16_t* L = static_cast<const bf16_t*>(p.latent) + b * p.l_sb;
  auto load_tile = [&](int c0) {
#pragma unroll
    for (int j = 0; j < NK; ++j) {
      const int i0 = 256 * j + 64 * wave, i = i0 + lane, n = i / NV;
      const int c = (i % NV) ^ img_f(n);  // source chunk of this position; past the row: any (times q = 0)
      const bf16_t* src = L + static_cast<int64_t>(min(c0 + n, k1 - 1)) * p.l_st + (8 * c < lq ? 8 * c : 0);
      __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)src,
                                       (__attribute__((address_space(3))) void*)(ls + 8 * i0), 16, 0, 0);
    }
  };
  if (k0 < k1) load_tile(k0);
  s16x8 qf[NK];
  {
    const bf16_t* Q = static_cast<const bf16_t*>(p.qcat) + (static_cast<int64_t>(b) * p.H + h0 + min(r, nh - 1)) * lq;
#pragma unroll
    for (int k = 0; k < NK; ++k) {
      const int d = 32 * k + 8 * g;
      bf16x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
      if (d < lq) v = load_bf16x8(Q + d);
      qf[k] = __builtin_bit_cast(s16x8, v);
    }
  }
  f32x4 acc[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m_run = -INFINITY, l_run = 0.f;  // of head 4 wave + g
  for (int c0 = k0; c0 < k1; c0 += kBN) {
    const int cnt = min(kBN, k1 - c0);
    if (c0 != k0) {
      __syncthreads();  // every wave is done with the last tile
      load_tile(c0);
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < NK; ++k)
      s = Mma<bf16_t>::mma(qf[k], Mma<bf16_t>::row(ls + img<NV>(16 * wave + r, 4 * k + g)), s);
#pragma unroll
    for (int i = 0; i < 4; ++i)
      ss[(4 * g + i) * kSS + 16 * wave + r] = 16 * wave + r < cnt ? s[i] * (p.scale * kLog2e) : -INFINITY;
    __syncthreads();
    {
      const float* row = ss + (4 * wave + g) * kSS + r;
      const float x[4] = {row[0], row[16], row[32], row[48]};
      __builtin_amdgcn_wave_barrier();  // (a row's 16 lanes have read it before any of them writes)
      float mx = fmaxf(fmaxf(x[0], x[1]), fmaxf(x[2], x[3]));
#pragma unroll
      for (int o = 1; o < 16; o <<= 1) mx = fmaxf(mx, __shfl_xor(mx, o, 64));
      const float mn = fmaxf(m_run, mx), mu = mn == -INFINITY ? 0.f : mn;
      const float a = exp2f(m_run - mu);
      m_run = mn;
      float l = 0.f;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float e = exp2f(x[j] - mu);
        l += e;
        put_planes<bf16_t>(ps + (4 * wave + g) * kSP + 16 * j + r, kBN, e);
      }
#pragma unroll
      for (int o = 1; o < 16; o <<= 1) l += __shfl_xor(l, o, 64);
      l_run = l_run * a + l;
      if (r == 0) al[4 * wave + g] = a;
    }
    __syncthreads();
    s16x8 ph[2], pl[2];
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      ph[k] = Mma<bf16_t>::row(ps + r * kSP + 32 * k + 8 * g);
      pl[k] = Mma<bf16_t>::row(ps + r * kSP + kBN + 32 * k + 8 * g);
    }
    float a4[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) a4[i] = al[4 * g + i];
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const int v0 = 16 * (wave + 4 * t);  // (columns past R are zeros or the rotated part: not stored)
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[t][i] *= a4[i];
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const int n = 32 * k + 8 * g + ((lane & 15) >> 2), ch = (v0 >> 3) + ((lane & 3) >> 1);
        const s16x4 a = tr4(ls + img<NV>(n, ch) + 4 * (lane & 1)), c = tr4(ls + img<NV>(n + 4, ch) + 4 * (lane & 1));
        const s16x8 bv = {a[0], a[1], a[2], a[3], c[0], c[1], c[2], c[3]};
        acc[t] = Mma<bf16_t>::mma(ph[k], bv, acc[t]);
        acc[t] = Mma<bf16_t>::mma(pl[k], bv, acc[t]);
      }
    }
  }
  const int64_t pb = (static_cast<int64_t>(b) * p.H + h0) * p.ns + split;
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int v = 16 * (wave + 4 * t) + r;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (v < p.R && 4 * g + i < nh) p.part_o[(pb + static_cast<int64_t>(4 * g + i) * p.ns) * p.R + v] = acc[t][i];
  }
  const int hh = 4 * wave + g;
  if (r == 0 && hh < nh) {
    p.part_ml[(pb + static_cast<int64_t>(hh) * p.ns) * 2] = m_run;
    p.part_ml[(pb + static_cast<int64_t>(hh) * p.ns) * 2 + 1] = l_run;
  }
}

template <int NK, int NT>
void go(const LatentParams& p, hipStream_t st) {
  constexpr int lds = 2 * kBN * 32 * NK + 4 * (16 * kSS + 16);
  if (lds > 64 * 1024)
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(latent_decode_mfma_kernel<NK, NT>),
                              hipFuncAttributeMaxDynamicSharedMemorySize, lds);
  latent_decode_mfma_kernel<NK, NT><<<dim3(p.ns, (p.H + 15) / 16, p.B), 256, lds, st>>>(p);
}

}  // namespace

bool latent_decode_mfma_ok(const LatentParams& p) {
  return p.R <= 512 && p.R + p.rot <= 576 && (p.R + p.rot) % 8 == 0 && p.l_st % 8 == 0 && p.l_sb % 8 == 0 &&
         reinterpret_cast<uintptr_t>(p.latent) % 16 == 0 && reinterpret_cast<uintptr_t>(p.qcat) % 16 == 0;
}

void launch_latent_decode_mfma(const LatentParams& p, hipStream_t st) {
  const int w = p.R + p.rot;
  if (w <= 192 && p.R <= 128) go<6, 2>(p, st);
  else if (w <= 320 && p.R <= 256) go<10, 4>(p, st);
  else go<18, 8>(p, st);
}

}  // namespace dla
