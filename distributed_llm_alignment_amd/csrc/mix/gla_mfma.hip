// Gated linear attention prefill on bf16 MFMA 32x32x16, chunks of 128 tokens in 4 sub-chunks of 32 (head
// sizes up to 256, multiples of 8; the rest: gla.hip). Four launches:
//
//   decay   l_t = log2 decay since the start of token t's sub-chunk (inclusive), per key channel; the
//           chunk's total
//   state   W[c] = V^T K' of chunk c, K'_s = k_s 2^(decays after s)       workgroup: 128 value rows x dim
//   scan    start state of every chunk: S <- 2^total S + W
//   output  workgroup = chunk, wave = sub-chunk, lane = token (all products transposed, so the scores'
//           accumulator is the next operand and the norm is in-lane plus one xor-32 step):
//             O^T  = S_start (q_t 2^(decays up to t))
//             O^T += V^T (K~ Q~^T)   per sub-chunk of keys up to the token's own
//
// A score needs q_t k_s 2^(decays in (s, t]) summed over channels. With e_j the total of sub-chunk j the
// decay is l_t + (e of the sub-chunks between) + (e_j - l_s): keys are staged once as k_s 2^(e_j - l_s),
// queries carry 2^(l_t + between), and no factor exceeds one however fast the decays are. In a token's
// own sub-chunk the query's factor is 2^(l_t - e_j), which is at least one: below 2^96 it is exact in the
// two planes; a (chunk, head) with a faster decay than that sums those scores channel by channel instead.
// Decayed q / k, scores and the state are fp32 values: hi + lo bf16 planes (mma.h).
#include "mix_params.h"
#include "mma.h"

namespace dla {
namespace {

constexpr int kC = 128, kSub = 32, kBN = 64, kThreads = 256;
constexpr float kFast = -96.f;  // the fastest sub-chunk decay (log2) the planes take
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

// log2(sigmoid(z)) = min(z, 0) log2 e - log2(1 + e^-|z|); with u = 1 + x rounded, log(1 + x) = log(u) x / (u - 1)
__device__ __forceinline__ float log2_sigmoid(float z) {
  constexpr float kLog2e = 1.4426950408889634f;
  const float x = __builtin_amdgcn_exp2f(-fabsf(z) * kLog2e), u = 1.f + x, d = u - 1.f;
  const float l = d == 0.f ? x * kLog2e : __builtin_amdgcn_logf(u) * (x * __builtin_amdgcn_rcpf(d));
  return fminf(z, 0.f) * kLog2e - l;
}

// grid (nc, ceil(H dim / 64), B), 4 waves: wave = sub-chunk of tokens, 2 tiles of 32 channels
__global__ __launch_bounds__(kThreads) void gla_decay_kernel(GlaParams p) {
  __shared__ float tot[4][64];
  const int b = blockIdx.z, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, Hd = p.H * p.dim, c32 = lane & 31, g = lane >> 5;
  const int t0 = blockIdx.x * kC + wave * kSub, kv0 = p.kv_start ? p.kv_start[b] : 0;
  const int64_t row0 = static_cast<int64_t>(b) * p.T;
  const bf16_t* A = static_cast<const bf16_t*>(p.proj) + (row0 + min(t0 + c32, p.T - 1)) * p.ld + 2 * (Hd + p.H * p.vdim);
  const bf16_t* W = static_cast<const bf16_t*>(p.a2);
  f32x16 z[2];
  float bias[2];
#pragma unroll
  for (int n = 0; n < 2; ++n) {
    bias[n] = bf2f(static_cast<const bf16_t*>(p.a2_b)[min(static_cast<int>(blockIdx.y) * 64 + 32 * n + c32, Hd - 1)]);
#pragma unroll
    for (int i = 0; i < 16; ++i) z[n][i] = 0.f;
  }
  for (int k0 = 0; k0 < p.rank; k0 += 16) {  // (rank % 8 == 0)
    const int k = k0 + 8 * g;
    const bool in = k < p.rank;
    s16x8 a = Mma<bf16_t>::zero(), w[2] = {a, a};
    if (in) {
      a = Mma<bf16_t>::row(A + k);
#pragma unroll
      for (int n = 0; n < 2; ++n)
        w[n] = Mma<bf16_t>::row(W + static_cast<int64_t>(min(static_cast<int>(blockIdx.y) * 64 + 32 * n + c32, Hd - 1)) * p.rank + k);
    }
#pragma unroll
    for (int n = 0; n < 2; ++n) z[n] = mfma32(a, w[n], z[n]);
  }
#pragma unroll
  for (int n = 0; n < 2; ++n) {
    const int ch = blockIdx.y * 64 + 32 * n + c32;
    // this lane's tokens are 8 u + 4 g + e: sums inside its groups of 4, then over both lanes' groups
    float before = 0.f;
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      float l[4], s = 0.f;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = t0 + 8 * u + 4 * g + e;
        if (t < p.T && p.base + t >= kv0) s += log2_sigmoid(z[n][4 * u + e] + bias[n]) * p.inv_tau;
        l[e] = s;
      }
      const float o = __shfl_xor(s, 32, 64), at = before + (g ? o : 0.f);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = t0 + 8 * u + 4 * g + e;
        if (t < p.T && ch < Hd) p.cum[(row0 + t) * Hd + ch] = at + l[e];
      }
      before += s + o;
    }
    if (g == 0) tot[wave][32 * n + c32] = before;
  }
  __syncthreads();
  const int ch = blockIdx.y * 64 + lane;
  if (wave == 0 && ch < Hd)
    p.total[(static_cast<int64_t>(b) * p.nc + blockIdx.x) * Hd + ch] = tot[0][lane] + tot[1][lane] + tot[2][lane] + tot[3][lane];
}

struct Head {
  int b, h, kv0, t0, len, Hd;
  const bf16_t* in;  // the chunk's rows
  const float* cum;  // the chunk's decays of this head
};
__device__ __forceinline__ Head head_of(const GlaParams& p, int c, int h, int b) {
  Head x{b, h, p.kv_start ? p.kv_start[b] : 0, c * kC, min(kC, p.T - c * kC), p.H * p.dim, nullptr, nullptr};
  const int64_t row = static_cast<int64_t>(b) * p.T + x.t0;
  x.in = static_cast<const bf16_t*>(p.proj) + row * p.ld;
  x.cum = p.cum + row * x.Hd + h * p.dim;
  return x;
}
// total log2 decay of sub-chunk j, channel d (0 past the end)
__device__ __forceinline__ float sub_total(const GlaParams& p, const Head& x, int j, int d) {
  const int t = min((j + 1) * kSub, x.len) - 1;
  return t >= j * kSub && d < p.dim ? x.cum[static_cast<int64_t>(t) * x.Hd + d] : 0.f;
}
// 8 channels of the decayed key of token t (zero past the end and in padding): k 2^(end[d] - l_t[d])
__device__ __forceinline__ void key8(const GlaParams& p, const Head& x, int t, int d, const float* end, float* v) {
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] = 0.f;
  if (t >= x.len || d >= p.dim || p.base + x.t0 + t < x.kv0) return;
  float l[8];
  load_vec<bf16_t, 8>(x.in + t * p.ld + x.Hd + x.h * p.dim + d, v);
  load_vec<float, 8>(x.cum + static_cast<int64_t>(t) * x.Hd + d, l);
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] *= __builtin_amdgcn_exp2f(end[d + e] - l[e]);
}
__device__ __forceinline__ bf16x8 value8(const GlaParams& p, const Head& x, int t, int v) {
  bf16x8 r = {0, 0, 0, 0, 0, 0, 0, 0};
  if (t < x.len && v < p.vdim && p.base + x.t0 + t >= x.kv0) r = load_bf16x8(x.in + t * p.ld + 2 * x.Hd + x.h * p.vdim + v);
  return r;
}

// grid (nc * ceil(vdim / 128), H, B): wave w = value rows 32 w .. + 31 of the block, all of dim
template <int ND>
__global__ __launch_bounds__(kThreads, ND > 4 ? 1 : 2) void gla_state_kernel(GlaParams p) {
  constexpr int DW = 32 * ND, SK = tr_stride(DW), SV = tr_stride(128), CK = DW / 8;
  __shared__ __attribute__((aligned(16))) bf16_t ks[2][kBN * SK];
  __shared__ __attribute__((aligned(16))) bf16_t vs[kBN * SV];
  __shared__ float after[4][DW];  // decay of sub-chunk j and what follows it in the chunk
  const int c = blockIdx.x % p.nc, vb = blockIdx.x / p.nc * 128;
  const Head x = head_of(p, c, blockIdx.y, blockIdx.z);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, c32 = lane & 31, g = lane >> 5;
  for (int d = threadIdx.x; d < DW; d += kThreads) {
    float s = 0.f;
#pragma unroll
    for (int j = 3; j >= 0; --j) {
      s += sub_total(p, x, j, d);
      after[j][d] = s;
    }
  }
  f32x16 acc[ND];
#pragma unroll
  for (int n = 0; n < ND; ++n)
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[n][i] = 0.f;
  for (int s0 = 0; s0 < x.len; s0 += kBN) {
    __syncthreads();
    for (int i = threadIdx.x; i < kBN * CK; i += kThreads) {
      const int t = i / CK, d = (i % CK) * 8;
      float v[8];
      key8(p, x, s0 + t, d, after[(s0 + t) / kSub], v);
      s16x8 hi, lo;
      Mma<bf16_t>::split(v, hi, lo);
      store_bf16x8(&ks[0][t * SK + d], __builtin_bit_cast(bf16x8, hi));
      store_bf16x8(&ks[1][t * SK + d], __builtin_bit_cast(bf16x8, lo));
    }
    for (int i = threadIdx.x; i < kBN * 16; i += kThreads) {
      const int t = i >> 4, v = (i & 15) * 8;
      store_bf16x8(vs + t * SV + v, value8(p, x, s0 + t, vb + v));
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
  float* W = p.work + ((static_cast<int64_t>(x.b) * p.H + x.h) * p.nc + c) * p.vdim * p.dim;
#pragma unroll
  for (int n = 0; n < ND; ++n)
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int v = vb + wave * 32 + 8 * (i >> 2) + 4 * g + (i & 3), d = 32 * n + c32;
      if (v < p.vdim && d < p.dim) W[static_cast<int64_t>(v) * p.dim + d] = acc[n][i];
    }
}

// grid (ceil(vdim dim / 4 / 256), H, B): work[c] <- start state of chunk c; state <- final state (dim % 4 == 0)
__global__ __launch_bounds__(256) void gla_scan_kernel(GlaParams p) {
  const int64_t n = static_cast<int64_t>(p.vdim) * p.dim;
  const int64_t i = (blockIdx.x * 256ll + threadIdx.x) * 4;
  if (i >= n) return;
  const int64_t bh = static_cast<int64_t>(blockIdx.z) * p.H + blockIdx.y, Hd = static_cast<int64_t>(p.H) * p.dim;
  float* st = p.state + bh * n + i;
  float* W = p.work + bh * p.nc * n + i;
  const float* D = p.total + static_cast<int64_t>(blockIdx.z) * p.nc * Hd + blockIdx.y * p.dim + i % p.dim;
  float s[4] = {0.f, 0.f, 0.f, 0.f};
  if (!p.fresh) load_vec<float, 4>(st, s);
  constexpr int U = 8;
  for (int c0 = 0; c0 < p.nc; c0 += U) {
    float w[U][4], f[U][4];
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (c0 + u < p.nc) {
        load_vec<float, 4>(W + (c0 + u) * n, w[u]);
        load_vec<float, 4>(D + (c0 + u) * Hd, f[u]);
      }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (c0 + u >= p.nc) break;
      store_vec<float, 4>(W + (c0 + u) * n, s);
#pragma unroll
      for (int e = 0; e < 4; ++e) s[e] = __builtin_amdgcn_exp2f(f[u][e]) * s[e] + w[u][e];
    }
  }
  store_vec<float, 4>(st, s);
}

// grid (nc, H, B). NK: 16-wide steps over dim, NV: 32-wide value tiles
template <int NK, int NV>
__global__ __launch_bounds__(kThreads, NK > 8 || NV > 4 ? 1 : 2) void gla_output_kernel(GlaParams p) {
  constexpr int DW = 16 * NK, SK = row_stride(DW), SV = tr_stride(32 * NV), CK = 2 * NK, CV = 4 * NV;
  __shared__ __attribute__((aligned(16))) bf16_t ks[2][kBN * SK];
  __shared__ __attribute__((aligned(16))) bf16_t vs[kBN * SV];
  __shared__ float sub[4][DW];   // log2 total of each sub-chunk
  __shared__ float fac[11][DW];  // query factors: 0-3 chunk start .. sub-chunk i, 4-6 between (2,0) (3,0) (3,1), 7-10 own
  __shared__ int fast;           // 0: some channel's decay is too fast for the planes
  const Head x = head_of(p, blockIdx.x, blockIdx.y, blockIdx.z);
  const int Hv = p.H * p.vdim;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, c32 = lane & 31, g = lane >> 5;
  const int tq = wave * 32 + c32;  // this lane's token in the chunk
  if (threadIdx.x == 0) fast = 1;
  __syncthreads();
  for (int d = threadIdx.x; d < DW; d += kThreads) {
    float e[4];
    bool ok = true;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      sub[j][d] = e[j] = sub_total(p, x, j, d);
      fac[7 + j][d] = exp2f(-fmaxf(e[j], kFast));
      ok = ok && e[j] >= kFast;
    }
    fac[0][d] = 1.f;
    fac[1][d] = exp2f(e[0]);
    fac[2][d] = exp2f(e[0] + e[1]);
    fac[3][d] = exp2f(e[0] + e[1] + e[2]);
    fac[4][d] = exp2f(e[1]);
    fac[5][d] = exp2f(e[1] + e[2]);
    fac[6][d] = exp2f(e[2]);
    if (!ok) fast = 0;
  }
  // q 2^(l_t) as planes
  s16x8 qh[NK], ql[NK];
#pragma unroll
  for (int s = 0; s < NK; ++s) {
    const int d = 16 * s + 8 * g;
    float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (tq < x.len && d < p.dim) {
      float l[8];
      load_vec<bf16_t, 8>(x.in + tq * p.ld + x.h * p.dim + d, v);
      load_vec<float, 8>(x.cum + static_cast<int64_t>(tq) * x.Hd + d, l);
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] *= p.qscale * __builtin_amdgcn_exp2f(l[e]);
    }
    Mma<bf16_t>::split(v, qh[s], ql[s]);
  }
  // step s of the query times factor row f
  auto scaled = [&](int s, const float* f, s16x8& h, s16x8& l) {
    float v[8];
#pragma unroll
    for (int e = 0; e < 8; ++e)
      v[e] = (bf2f(static_cast<bf16_t>(qh[s][e])) + bf2f(static_cast<bf16_t>(ql[s][e]))) * f[16 * s + 8 * g + e];
    Mma<bf16_t>::split(v, h, l);
  };
  f32x16 o[NV];
#pragma unroll
  for (int t = 0; t < NV; ++t)
#pragma unroll
    for (int i = 0; i < 16; ++i) o[t][i] = 0.f;
  __syncthreads();
  if (!p.fresh || blockIdx.x > 0) {  // (chunk 0 of a fresh sequence starts at zero)
    const float* S = p.work + ((static_cast<int64_t>(x.b) * p.H + x.h) * p.nc + blockIdx.x) * p.vdim * p.dim;
#pragma unroll
    for (int s = 0; s < NK; ++s) {
      const int d = 16 * s + 8 * g;
      s16x8 ah, al;
      scaled(s, fac[wave], ah, al);
#pragma unroll
      for (int t = 0; t < NV; ++t) {
        const int v = 32 * t + c32;
        float y[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
        if (d < p.dim && v < p.vdim) load_vec<float, 8>(S + static_cast<int64_t>(v) * p.dim + d, y);
        s16x8 sh, sl;
        Mma<bf16_t>::split(y, sh, sl);
        o[t] = mfma32(sh, ah, o[t]);
        o[t] = mfma32(sl, ah, o[t]);
        o[t] = mfma32(sh, al, o[t]);
      }
    }
  }
  for (int s0 = 0; s0 < x.len; s0 += kBN) {
    __syncthreads();
    for (int i = threadIdx.x; i < kBN * CK; i += kThreads) {
      const int t = i / CK, d = (i % CK) * 8;
      float v[8];
      key8(p, x, s0 + t, d, sub[(s0 + t) / kSub], v);
      s16x8 hi, lo;
      Mma<bf16_t>::split(v, hi, lo);
      store_bf16x8(&ks[0][t * SK + d], __builtin_bit_cast(bf16x8, hi));
      store_bf16x8(&ks[1][t * SK + d], __builtin_bit_cast(bf16x8, lo));
    }
    for (int i = threadIdx.x; i < kBN * CV; i += kThreads) {
      const int t = i / CV, v = (i % CV) * 8;
      store_bf16x8(vs + t * SV + v, value8(p, x, s0 + t, v));
    }
    __syncthreads();
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      const int j = s0 / kSub + n;  // this sub-chunk of keys against the wave's sub-chunk of queries
      if (j > wave) continue;
      f32x16 s;
#pragma unroll
      for (int i = 0; i < 16; ++i) s[i] = 0.f;
      if (j < wave || fast) {
        const float* f = j == wave ? fac[7 + j] : wave - j == 1 ? fac[0] : j == 1 ? fac[6] : wave == 2 ? fac[4] : fac[5];
#pragma unroll
        for (int k = 0; k < NK; ++k) {
          const s16x8 kh = __builtin_bit_cast(s16x8, load_bf16x8(&ks[0][(32 * n + c32) * SK + 16 * k + 8 * g]));
          const s16x8 kl = __builtin_bit_cast(s16x8, load_bf16x8(&ks[1][(32 * n + c32) * SK + 16 * k + 8 * g]));
          s16x8 ah = qh[k], al = ql[k];
          if (wave - j != 1) scaled(k, f, ah, al);
          s = mfma32(kh, ah, s);
          s = mfma32(kl, ah, s);
          s = mfma32(kh, al, s);
        }
      } else {
        // too fast a decay for the planes: every (token, key) pair by itself
#pragma unroll 1
        for (int i = 0; i < 16; ++i) {
          const int tk = j * kSub + 8 * (i >> 2) + 4 * g + (i & 3);
          float v = 0.f;
          if (tk <= tq && tq < x.len && p.base + x.t0 + tk >= x.kv0) {
            const bf16_t *qr = x.in + tq * p.ld + x.h * p.dim, *kr = x.in + tk * p.ld + x.Hd + x.h * p.dim;
            const float *lq = x.cum + static_cast<int64_t>(tq) * x.Hd, *lk = x.cum + static_cast<int64_t>(tk) * x.Hd;
            for (int d = 0; d < p.dim; ++d) v += bf2f(qr[d]) * bf2f(kr[d]) * __builtin_amdgcn_exp2f(lq[d] - lk[d]);
          }
#pragma unroll
          for (int e = 0; e < 16; ++e) s[e] = e == i ? v * p.qscale : s[e];
        }
      }
      if (j == wave) {
#pragma unroll
        for (int i = 0; i < 16; ++i)
          if (j * kSub + 8 * (i >> 2) + 4 * g + (i & 3) > tq) s[i] = 0.f;
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
  if (tq >= x.len) return;
  const float rs = rsqrtf(ss / p.vdim + p.eps);
  const bf16_t* gr = x.in + tq * p.ld + 2 * x.Hd + Hv + x.h * p.vdim;
  const bf16_t* nw = static_cast<const bf16_t*>(p.norm_w);
  bf16_t* yr = static_cast<bf16_t*>(p.y) + (static_cast<int64_t>(x.b) * p.T + x.t0 + tq) * Hv + x.h * p.vdim;
#pragma unroll
  for (int t = 0; t < NV; ++t)
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int v = 32 * t + 8 * u + 4 * g;
      if (v >= p.vdim) continue;
      const bf16x4 gv = *reinterpret_cast<const bf16x4*>(gr + v), wv = *reinterpret_cast<const bf16x4*>(nw + v);
      float y[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float z = bf2f(gv[e]);
        y[e] = o[t][4 * u + e] * rs * bf2f(wv[e]) * (z / (1.f + __expf(-z)));
      }
      typedef uint32_t u32x2 __attribute__((ext_vector_type(2)));
      *reinterpret_cast<u32x2*>(yr + v) = u32x2{pack2bf(y[0], y[1]), pack2bf(y[2], y[3])};
    }
}

}  // namespace

// chunks of the chunked form, 0: the recurrence takes the portion
int gla_chunks(bool bf16, const GlaParams& p) {
  const auto al = [](const void* x) { return reinterpret_cast<uintptr_t>(x) % 16 == 0; };
  const bool ok = bf16 && p.T >= 16 && p.dim % 8 == 0 && p.vdim % 8 == 0 && p.ld % 8 == 0 && p.dim <= 256 && p.vdim <= 256 &&
                  al(p.proj) && al(p.y) && al(p.norm_w) && al(p.a2);
  return ok ? (p.T + kC - 1) / kC : 0;
}

void launch_gla_prefill(const GlaParams& p, hipStream_t st) {
  const int Hd = p.H * p.dim;
  const int64_t n = static_cast<int64_t>(p.vdim) * p.dim;
  gla_decay_kernel<<<dim3(p.nc, (Hd + 63) / 64, p.B), kThreads, 0, st>>>(p);
  const dim3 gs(p.nc * ((p.vdim + 127) / 128), p.H, p.B);
  if (p.dim <= 64) gla_state_kernel<2><<<gs, kThreads, 0, st>>>(p);
  else if (p.dim <= 128) gla_state_kernel<4><<<gs, kThreads, 0, st>>>(p);
  else gla_state_kernel<8><<<gs, kThreads, 0, st>>>(p);
  gla_scan_kernel<<<dim3((n / 4 + 255) / 256, p.H, p.B), 256, 0, st>>>(p);
  const dim3 go(p.nc, p.H, p.B);
  if (p.dim <= 64 && p.vdim <= 64) gla_output_kernel<4, 2><<<go, kThreads, 0, st>>>(p);
  else if (p.dim <= 128 && p.vdim <= 128) gla_output_kernel<8, 4><<<go, kThreads, 0, st>>>(p);
  else if (p.dim <= 128) gla_output_kernel<8, 8><<<go, kThreads, 0, st>>>(p);
  else gla_output_kernel<16, 8><<<go, kThreads, 0, st>>>(p);
}

}  // namespace dla
