// Latent attention for gfx950: heads' keys and values are projections of one cached latent per token
// plus one rotated key part shared by all heads; softmax over a sliding window.
//
//   prepare   per token: RMS norms of the query latent and of the cached latent, rotation of the
//             shared key part, cache write
//   prefill   flash attention over up-projected keys / values (any head sizes, bf16 or fp32; the
//             bf16 sizes of latent_prefill.hip take that kernel instead)
//   absorb    decode: query heads into latent space (q W_uk), rotated part appended
//   decode    split-key attention on the latent cache, all heads of a group share each key tile
//   combine   merge of the splits and W_uv
//
// Columns below kv_start[b] are padding; a token's position is its column - kv_start[b]. Query column
// i sees key column j iff kv_start <= j <= i and (window == 0 or i - j < window). Scores, softmax
// weights (hi + lo planes on bf16 MFMAs) and all sums are fp32.
#include "mix_params.h"
#include "mma.h"

namespace dla {

bool latent_decode_mfma_ok(const LatentParams&);  // latent_decode.hip
void launch_latent_decode_mfma(const LatentParams&, hipStream_t);

namespace {

constexpr float kLog2e = 1.4426950408889634f;
constexpr int kLdsMax = 160 * 1024;

template <typename T>
constexpr int pad16() { return 16 / static_cast<int>(sizeof(T)); }

template <typename K>
void allow_lds(K kernel, int64_t bytes) {
  if (bytes > 64 * 1024)
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize,
                              static_cast<int>(bytes));
}

// ------------------------------------------------------------------------------------ prepare
// One workgroup per token. down row: [q latent (qr) | kv latent (R) | key part (rot)].
template <typename T, int VEC>
__global__ __launch_bounds__(128) void latent_prepare_kernel(
    const T* __restrict__ down, int64_t ld, const T* __restrict__ qw, const T* __restrict__ kw, float eps,
    T* __restrict__ cq, T* __restrict__ latent, int64_t l_sb, int64_t l_st, const int64_t* __restrict__ slot,
    const int* __restrict__ kv_start, const float* __restrict__ cos_t, const float* __restrict__ sin_t, int Tn,
    int qr, int R, int rot, int tcap) {
  __shared__ float scratch[2];
  const int64_t row = blockIdx.x;
  const int b = static_cast<int>(row / Tn), t = static_cast<int>(row % Tn);
  const int64_t col = min(slot[0] + t, static_cast<int64_t>(tcap - 1));  // (a full cache is the host's error)
  const T* in = down + row * ld;
  T* out = latent + b * l_sb + col * l_st;
  float sq = 0.f, sk = 0.f, v[VEC], w[VEC];
  for (int i = threadIdx.x * VEC; i < qr; i += 128 * VEC) {
    load_vec<T, VEC>(in + i, v);
#pragma unroll
    for (int e = 0; e < VEC; ++e) sq += v[e] * v[e];
  }
  for (int i = threadIdx.x * VEC; i < R; i += 128 * VEC) {
    load_vec<T, VEC>(in + qr + i, v);
#pragma unroll
    for (int e = 0; e < VEC; ++e) sk += v[e] * v[e];
  }
  const float rq = rsqrtf(block_sum<128>(sq, scratch) / qr + eps);
  const float rk = rsqrtf(block_sum<128>(sk, scratch) / R + eps);
  for (int i = threadIdx.x * VEC; i < qr; i += 128 * VEC) {
    load_vec<T, VEC>(in + i, v);
    load_vec<T, VEC>(qw + i, w);
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = v[e] * rq * w[e];
    store_vec<T, VEC>(cq + row * qr + i, v);
  }
  for (int i = threadIdx.x * VEC; i < R; i += 128 * VEC) {
    load_vec<T, VEC>(in + qr + i, v);
    load_vec<T, VEC>(kw + i, w);
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = v[e] * rk * w[e];
    store_vec<T, VEC>(out + i, v);
  }
  const int64_t pos = max(col - (kv_start ? kv_start[b] : 0), static_cast<int64_t>(0));
  for (int i = threadIdx.x; i < rot; i += 128) {
    float r;
    load_rotated<T, 1>(in + qr + R, i, rot, cos_t + pos * (rot >> 1), sin_t + pos * (rot >> 1), &r);
    out[R + i] = from_f<T>(r);
  }
}

// ------------------------------------------------------------------------------------ prefill
// grid (query blocks, H, B), NW waves of 16 queries each; key tiles of 32.
template <typename T>
__global__ __launch_bounds__(256) void latent_prefill_any_kernel(LatentParams p) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  using M = Mma<T>;
  constexpr int BN = 32;
  const int NW = blockDim.x >> 6, BM = 16 * NW;
  const int h = blockIdx.y, b = blockIdx.z, q0 = blockIdx.x * BM;
  const int dq = p.dim + p.rot, dp = round_up(dq, 32), vp = round_up(p.vdim, 16);
  const int ldq = dp + pad16<T>(), ldv = vp + pad16<T>(), ldp = BN + pad16<T>(), ldo = vp + 4;
  T* qs = reinterpret_cast<T*>(smem);
  T* ks = qs + BM * ldq;
  T* vs = ks + BN * ldq;
  T* ps = vs + BN * ldv;
  float* os = reinterpret_cast<float*>(ps + NW * M::PL * 16 * ldp);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane & 15, g = lane >> 4;
  const int kv0 = p.kv_start ? p.kv_start[b] : 0, half = p.rot >> 1;
  const T* Q = static_cast<const T*>(p.q) + static_cast<int64_t>(b) * p.T * p.H * dq + h * dq;
  const int ldkv = p.H * (p.dim + p.vdim);
  const T* KV = static_cast<const T*>(p.kv) + static_cast<int64_t>(b) * p.S * ldkv;
  const T* KR = static_cast<const T*>(p.kr) + b * p.kr_sb;
  for (int i = threadIdx.x; i < BM * dp; i += blockDim.x) {
    const int m = i / dp, d = i % dp, t = q0 + m;
    float v = 0.f;
    if (t < p.T && d < dq) {
      const T* row = Q + static_cast<int64_t>(t) * p.H * dq;
      if (d < p.dim) {
        v = to_f<T>(row[d]);
      } else {
        const int64_t pos = max(p.q_base + t - kv0, 0);
        load_rotated<T, 1>(row + p.dim, d - p.dim, p.rot, p.cos_t + pos * half, p.sin_t + pos * half, &v);
      }
    }
    qs[m * ldq + d] = from_f<T>(v);
  }
  for (int i = threadIdx.x; i < BM * ldo; i += blockDim.x) os[i] = 0.f;
  // this lane's 4 query rows
  float m_run[4], l_run[4];
  int qc[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    m_run[i] = -INFINITY;
    l_run[i] = 0.f;
    qc[i] = p.q_base + q0 + wave * 16 + 4 * g + i;
  }
  int lo = max(kv0, p.k_base), hi = min(p.q_base + min(q0 + BM, p.T), p.k_base + p.S);
  if (p.window) lo = max(lo, p.q_base + q0 - p.window + 1);
  for (int c0 = lo; c0 < hi; c0 += BN) {
    __syncthreads();
    for (int i = threadIdx.x; i < BN * dp; i += blockDim.x) {
      const int n = i / dp, d = i % dp, s = c0 + n - p.k_base;
      T v = from_f<T>(0.f);
      if (s < p.S && d < dq) v = d < p.dim ? KV[static_cast<int64_t>(s) * ldkv + h * p.dim + d] : KR[s * p.kr_st + d - p.dim];
      ks[n * ldq + d] = v;
    }
    for (int i = threadIdx.x; i < BN * vp; i += blockDim.x) {
      const int n = i / vp, d = i % vp, s = c0 + n - p.k_base;
      vs[n * ldv + d] = s < p.S && d < p.vdim ? KV[static_cast<int64_t>(s) * ldkv + p.H * p.dim + h * p.vdim + d] : from_f<T>(0.f);
    }
    __syncthreads();
    f32x4 sc[2];
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      sc[n] = f32x4{0.f, 0.f, 0.f, 0.f};
      for (int k = 0; k < dp; k += M::KS)
        sc[n] = M::mma(M::row(qs + (wave * 16 + r) * ldq + k + g * M::KV), M::row(ks + (n * 16 + r) * ldq + k + g * M::KV), sc[n]);
    }
    T* pw = ps + wave * M::PL * 16 * ldp;
    float alpha[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      float mx = -INFINITY;
#pragma unroll
      for (int n = 0; n < 2; ++n) {
        const int j = c0 + n * 16 + r;
        const bool ok = j < hi && j <= qc[i] && (p.window == 0 || qc[i] - j < p.window);
        sc[n][i] = ok ? sc[n][i] * (p.scale * kLog2e) : -INFINITY;
        mx = fmaxf(mx, sc[n][i]);
      }
#pragma unroll
      for (int o = 1; o < 16; o <<= 1) mx = fmaxf(mx, __shfl_xor(mx, o, 64));
      const float mn = fmaxf(m_run[i], mx), mu = mn == -INFINITY ? 0.f : mn;
      alpha[i] = exp2f(m_run[i] - mu);
      m_run[i] = mn;
      float l = 0.f;
#pragma unroll
      for (int n = 0; n < 2; ++n) {
        const float e = exp2f(sc[n][i] - mu);
        l += e;
        put_planes<T>(pw + (4 * g + i) * ldp + n * 16 + r, 16 * ldp, e);
      }
      l_run[i] = l_run[i] * alpha[i] + l;  // per-lane partial (columns r); summed at the end
    }
    __syncthreads();
    for (int v0 = 0; v0 < vp; v0 += 16) {
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
      for (int k = 0; k < BN; k += M::KS) {
        const auto bv = M::col(vs + (k + g * M::KV) * ldv + v0 + r, ldv);
        const T* pp = pw + r * ldp + k + g * M::KV;
        acc = M::mma(M::row(pp), bv, acc);
        if constexpr (M::PL == 2) acc = M::mma(M::row(pp + 16 * ldp), bv, acc);
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        float* o = os + (wave * 16 + 4 * g + i) * ldo + v0 + r;
        *o = *o * alpha[i] + acc[i];
      }
    }
  }
  __syncthreads();  // (a block of padding queries ran no tile: its zeros come from other threads)
  T* O = static_cast<T*>(p.o) + static_cast<int64_t>(b) * p.T * p.H * p.vdim + h * p.vdim;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    float l = l_run[i];
#pragma unroll
    for (int o = 1; o < 16; o <<= 1) l += __shfl_xor(l, o, 64);
    const int m = wave * 16 + 4 * g + i, t = q0 + m;
    if (t >= p.T) continue;
    const float inv = l > 0.f ? 1.f / l : 0.f;
    for (int v = r; v < p.vdim; v += 16) O[static_cast<int64_t>(t) * p.H * p.vdim + v] = from_f<T>(os[m * ldo + v] * inv);
  }
}

template <typename T>
int64_t prefill_lds(const LatentParams& p, int NW) {
  const int dp = round_up(p.dim + p.rot, 32), vp = round_up(p.vdim, 16), pd = pad16<T>();
  return static_cast<int64_t>(sizeof(T)) * ((16 * NW + 32) * (dp + pd) + 32 * (vp + pd) + NW * Mma<T>::PL * 16 * (32 + pd)) +
         4ll * 16 * NW * (vp + 4);
}

template <typename T>
int prefill_waves(const LatentParams& p) {
  for (int nw = 4; nw >= 1; nw /= 2)
    if (prefill_lds<T>(p, nw) <= kLdsMax) return nw;
  return 0;
}

// ------------------------------------------------------------------------------------- absorb
// qcat[b][h] = [sum_d q[b][h][d] W_uk[h][d][:] | rotated q part]. grid (H, ceil(R / 64)), 256 threads:
// 8 column groups of 8 x 32 slices of d; batch rows in groups of 4.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void latent_absorb_kernel(LatentParams p) {
  __shared__ float red[32][4][66];
  const int h = blockIdx.x, r0 = blockIdx.y * 64;
  const int dq = p.dim + p.rot, lq = p.R + p.rot, half = p.rot >> 1;
  const int cg = threadIdx.x & 7, dg = threadIdx.x >> 3;
  const T* W = static_cast<const T*>(p.kv_up) + static_cast<int64_t>(h) * p.dim * p.R;
  const T* Q = static_cast<const T*>(p.q) + h * dq;
  T* out = static_cast<T*>(p.qcat) + static_cast<int64_t>(h) * lq;
  const int64_t qsb = static_cast<int64_t>(p.H) * dq, osb = static_cast<int64_t>(p.H) * lq;
  for (int b0 = 0; b0 < p.B; b0 += 4) {
    float acc[4][8];
#pragma unroll
    for (int b = 0; b < 4; ++b)
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[b][e] = 0.f;
    const int rc = r0 + cg * 8;
    for (int d = dg; d < p.dim; d += 32) {
      float w[8];
      if constexpr (VEC == 8) {
#pragma unroll
        for (int e = 0; e < 8; ++e) w[e] = 0.f;
        if (rc < p.R) load_vec<T, 8>(W + static_cast<int64_t>(d) * p.R + rc, w);
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e) w[e] = rc + e < p.R ? to_f<T>(W[static_cast<int64_t>(d) * p.R + rc + e]) : 0.f;
      }
#pragma unroll
      for (int b = 0; b < 4; ++b) {
        const float q = b0 + b < p.B ? to_f<T>(Q[(b0 + b) * qsb + d]) : 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[b][e] += q * w[e];
      }
    }
#pragma unroll
    for (int b = 0; b < 4; ++b)
#pragma unroll
      for (int e = 0; e < 8; ++e) red[dg][b][cg * 8 + e] = acc[b][e];
    __syncthreads();
    const int b = threadIdx.x >> 6, c = threadIdx.x & 63;
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < 32; ++j) s += red[j][b][c];
    if (b0 + b < p.B && r0 + c < p.R) out[(b0 + b) * osb + r0 + c] = from_f<T>(s);
    __syncthreads();
  }
  if (blockIdx.y == 0) {
    for (int i = threadIdx.x; i < p.B * p.rot; i += 256) {
      const int b = i / p.rot, d = i % p.rot;
      const int64_t pos = max(min(p.slot[0], static_cast<int64_t>(p.tcap - 1)) - (p.kv_start ? p.kv_start[b] : 0), static_cast<int64_t>(0));
      float v;
      load_rotated<T, 1>(Q + b * qsb + p.dim, d, p.rot, p.cos_t + pos * half, p.sin_t + pos * half, &v);
      out[b * osb + p.R + d] = from_f<T>(v);
    }
  }
}

// The same on MFMA (bf16, dim <= 256, dim, rot and R multiples of 8): the head's [dim, 64] piece of W_uk
// is staged as rows in LDS and read back transposed; wave w owns 16 of the 64 columns, batch rows
// ride on the MFMA's row dimension.
typedef __attribute__((address_space(3))) s16x4 lds_s16x4;
template <int ND>
__global__ __launch_bounds__(256) void latent_absorb_mfma_kernel(LatentParams p) {
  constexpr int SW = 64 + 24;  // row stride: odd multiple of 16 B, 4 rows' 32-byte pieces on distinct banks
  __shared__ __attribute__((aligned(16))) bf16_t ws[32 * ND * SW];
  const int h = blockIdx.x, r0 = blockIdx.y * 64;
  const int dq = p.dim + p.rot, lq = p.R + p.rot, half = p.rot >> 1;
  const bf16_t* W = static_cast<const bf16_t*>(p.kv_up) + static_cast<int64_t>(h) * p.dim * p.R;
  const bf16_t* Q = static_cast<const bf16_t*>(p.q) + h * dq;
  bf16_t* out = static_cast<bf16_t*>(p.qcat) + static_cast<int64_t>(h) * lq;
  const int64_t qsb = static_cast<int64_t>(p.H) * dq, osb = static_cast<int64_t>(p.H) * lq;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane & 15, g = lane >> 4;
  bf16x8 reg[ND];
#pragma unroll
  for (int j = 0; j < ND; ++j) {
    const int i = threadIdx.x + 256 * j, d = i >> 3, c = r0 + (i & 7) * 8;
    bf16x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
    if (d < p.dim && c < p.R) v = load_bf16x8(W + static_cast<int64_t>(d) * p.R + c);
    reg[j] = v;
  }
  s16x8 qf[ND];
  auto load_q = [&](int b0) {
#pragma unroll
    for (int k = 0; k < ND; ++k) {
      const int d = 32 * k + 8 * g;
      bf16x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
      if (d < p.dim) v = load_bf16x8(Q + min(b0 + r, p.B - 1) * qsb + d);
      qf[k] = __builtin_bit_cast(s16x8, v);
    }
  };
  load_q(0);
#pragma unroll
  for (int j = 0; j < ND; ++j) {
    const int i = threadIdx.x + 256 * j;
    store_bf16x8(ws + (i >> 3) * SW + (i & 7) * 8, reg[j]);
  }
  __syncthreads();
  for (int b0 = 0; b0 < p.B; b0 += 16) {
    if (b0) load_q(b0);
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < ND; ++k) {
      const bf16_t* wp = ws + (32 * k + 8 * g + ((lane & 15) >> 2)) * SW + 16 * wave + 4 * (lane & 3);
      const s16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)(wp));
      const s16x4 c = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)(wp + 4 * SW));
      acc = Mma<bf16_t>::mma(qf[k], s16x8{a[0], a[1], a[2], a[3], c[0], c[1], c[2], c[3]}, acc);
    }
    const int col = r0 + 16 * wave + r;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (b0 + 4 * g + i < p.B && col < p.R) out[(b0 + 4 * g + i) * osb + col] = f2bf(acc[i]);
  }
  if (blockIdx.y == 0) {
    for (int i = threadIdx.x; i < p.B * p.rot; i += 256) {
      const int b = i / p.rot, d = i % p.rot;
      const int64_t pos = max(min(p.slot[0], static_cast<int64_t>(p.tcap - 1)) - (p.kv_start ? p.kv_start[b] : 0), static_cast<int64_t>(0));
      float v;
      load_rotated<bf16_t, 1>(Q + b * qsb + p.dim, d, p.rot, p.cos_t + pos * half, p.sin_t + pos * half, &v);
      out[b * osb + p.R + d] = f2bf(v);
    }
  }
}

// ------------------------------------------------------------------------------------- decode
// grid (ns, ceil(H / 16), B), 256 threads; key tiles of BN (32 or 64); NT = latent column tiles per wave
template <typename T, int NT>
__global__ __launch_bounds__(256) void latent_decode_kernel(LatentParams p, int BN) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  using M = Mma<T>;
  const int split = blockIdx.x, h0 = blockIdx.y * 16, b = blockIdx.z;
  const int lq = p.R + p.rot, lp = round_up(lq, 32), ldl = lp + pad16<T>(), ldp = BN + pad16<T>();
  T* ls = reinterpret_cast<T*>(smem);
  T* ps = ls + BN * ldl;
  float* ss = reinterpret_cast<float*>(ps + M::PL * 16 * ldp);  // [16][BN + 1] scores
  float* al = ss + 16 * (BN + 1);                               // [16] rescale of this tile
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane & 15, g = lane >> 4;
  const int64_t newest = min(p.slot[0], static_cast<int64_t>(p.tcap - 1));
  int64_t lo = p.kv_start ? p.kv_start[b] : 0;
  if (p.window) lo = max(lo, newest - p.window + 1);
  const int64_t n = newest - lo + 1;
  int64_t per = (n + p.ns - 1) / p.ns;
  per = (per + BN - 1) / BN * BN;
  const int64_t k0 = lo + split * per, k1 = min(k0 + per, newest + 1);
  const T* L = static_cast<const T*>(p.latent) + b * p.l_sb;
  const T* Q = static_cast<const T*>(p.qcat) + (static_cast<int64_t>(b) * p.H + h0) * lq;
  const int nh = min(16, p.H - h0);
  f32x4 acc[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  // softmax: wave w owns heads 4w .. 4w+3, 16 lanes each
  float m_run = -INFINITY, l_run = 0.f;
  const bool vec = lq % 8 == 0 && p.l_st % 8 == 0 && p.l_sb % 8 == 0 && (reinterpret_cast<uintptr_t>(L) % 16) == 0 &&
                   (reinterpret_cast<uintptr_t>(Q) % 16) == 0;
  for (int64_t c0 = k0; c0 < k1; c0 += BN) {
    const int cnt = static_cast<int>(min(static_cast<int64_t>(BN), k1 - c0));
    __syncthreads();
    if (vec) {
      const int nv = lp / 8;
      for (int i = threadIdx.x; i < BN * nv; i += 256) {
        const int k = i / nv, d = (i % nv) * 8;
        if constexpr (sizeof(T) == 2) {
          bf16x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
          if (k < cnt && d < lq) v = load_bf16x8(reinterpret_cast<const bf16_t*>(L + (c0 + k) * p.l_st + d));
          store_bf16x8(reinterpret_cast<bf16_t*>(ls + k * ldl + d), v);
        } else {
          float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
          if (k < cnt && d < lq) load_vec<T, 8>(L + (c0 + k) * p.l_st + d, v);
          store_vec<T, 8>(ls + k * ldl + d, v);
        }
      }
    } else {
      for (int i = threadIdx.x; i < BN * lp; i += 256) {
        const int k = i / lp, d = i % lp;
        ls[k * ldl + d] = k < cnt && d < lq ? L[(c0 + k) * p.l_st + d] : from_f<T>(0.f);
      }
    }
    __syncthreads();
    for (int kt = wave; kt < BN / 16; kt += 4) {
      f32x4 s = {0.f, 0.f, 0.f, 0.f};
      for (int k = 0; k < lp; k += M::KS) {
        const int d = k + g * M::KV;
        auto a = M::zero();
        if (r < nh && d < lq) {
          const T* qp = Q + static_cast<int64_t>(r) * lq + d;
          if (vec) {
            a = M::row(qp);
          } else {
#pragma unroll
            for (int e = 0; e < M::KV; ++e)
              if (d + e < lq) M::set(a, e, qp[e]);
          }
        }
        s = M::mma(a, M::row(ls + (kt * 16 + r) * ldl + d), s);
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
        ss[(4 * g + i) * (BN + 1) + kt * 16 + r] = kt * 16 + r < cnt ? s[i] * (p.scale * kLog2e) : -INFINITY;
    }
    __syncthreads();
    {
      const int hh = 4 * wave + g;
      float mx = -INFINITY;
      for (int j = r; j < BN; j += 16) mx = fmaxf(mx, ss[hh * (BN + 1) + j]);
#pragma unroll
      for (int o = 1; o < 16; o <<= 1) mx = fmaxf(mx, __shfl_xor(mx, o, 64));
      const float mn = fmaxf(m_run, mx), mu = mn == -INFINITY ? 0.f : mn;
      const float a = exp2f(m_run - mu);
      m_run = mn;
      float l = 0.f;
      for (int j = r; j < BN; j += 16) {
        const float e = exp2f(ss[hh * (BN + 1) + j] - mu);
        l += e;
        put_planes<T>(ps + hh * ldp + j, 16 * ldp, e);
      }
#pragma unroll
      for (int o = 1; o < 16; o <<= 1) l += __shfl_xor(l, o, 64);
      l_run = l_run * a + l;
      if (r == 0) al[hh] = a;
    }
    __syncthreads();
    float a4[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) a4[i] = al[4 * g + i];
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const int v0 = (wave + 4 * t) * 16;
      if (v0 >= p.R) continue;
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[t][i] *= a4[i];
      for (int k = 0; k < BN; k += M::KS) {
        const auto bv = M::col(ls + (k + g * M::KV) * ldl + v0 + r, ldl);
        const T* pp = ps + r * ldp + k + g * M::KV;
        acc[t] = M::mma(M::row(pp), bv, acc[t]);
        if constexpr (M::PL == 2) acc[t] = M::mma(M::row(pp + 16 * ldp), bv, acc[t]);
      }
    }
  }
  const int64_t pb = (static_cast<int64_t>(b) * p.H + h0) * p.ns + split;
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int v = (wave + 4 * t) * 16 + r;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int hh = 4 * g + i;
      if (v < p.R && hh < nh) p.part_o[(pb + static_cast<int64_t>(hh) * p.ns) * p.R + v] = acc[t][i];
    }
  }
  const int hh = 4 * wave + g;
  if (r == 0 && hh < nh) {
    p.part_ml[(pb + static_cast<int64_t>(hh) * p.ns) * 2] = m_run;
    p.part_ml[(pb + static_cast<int64_t>(hh) * p.ns) * 2 + 1] = l_run;
  }
}

template <typename T>
int64_t decode_lds(const LatentParams& p, int BN) {
  const int lp = round_up(p.R + p.rot, 32), pd = pad16<T>();
  return static_cast<int64_t>(sizeof(T)) * (BN * (lp + pd) + Mma<T>::PL * 16 * (BN + pd)) + 4ll * (16 * (BN + 1) + 16);
}

// ------------------------------------------------------------------------------------ combine
// grid (H, B, ceil(vdim / kCombV)), 256 threads: o[b][h] = W_uv[h] (sum over splits). ns <= 256.
constexpr int kCombV = 32;
template <typename T, int VEC>
__global__ __launch_bounds__(256) void latent_combine_kernel(LatentParams p) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  float* os = reinterpret_cast<float*>(smem);  // [R]
  __shared__ float ws[256];
  __shared__ float scratch[4];
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x;
  const int64_t pb = (static_cast<int64_t>(b) * p.H + h) * p.ns;
  // independent of everything below: the first piece of this wave's W_uv rows, the first splits
  const T* W = static_cast<const T*>(p.kv_up) + (static_cast<int64_t>(p.H) * p.dim + static_cast<int64_t>(h) * p.vdim) * p.R;
  const int wave = tid >> 6, lane = tid & 63;
  constexpr int U = kCombV / 4;
  const int v0 = blockIdx.z * kCombV + wave * U;
  float wv[U][VEC];
  auto load_w = [&](int c) {
#pragma unroll
    for (int u = 0; u < U; ++u) load_vec<T, VEC>(W + static_cast<int64_t>(min(v0 + u, p.vdim - 1)) * p.R + c, wv[u]);
  };
  if (lane * VEC < p.R) load_w(lane * VEC);
  const float m = tid < p.ns ? p.part_ml[(pb + tid) * 2] : -INFINITY;
  const float l0 = tid < p.ns ? p.part_ml[(pb + tid) * 2 + 1] : 0.f;
  const float mx = block_max<256>(m, scratch);
  const float w = m == -INFINITY ? 0.f : exp2f(m - mx);
  const float l = block_sum<256>(w * l0, scratch);
  ws[tid] = l > 0.f ? w / l : 0.f;
  __syncthreads();
  for (int c = tid; c < p.R; c += 256) {
    float v = 0.f;
    int s = 0;
    for (; s + 16 <= p.ns; s += 16) {  // (empty splits hold zeros)
      float x[16];
#pragma unroll
      for (int u = 0; u < 16; ++u) x[u] = p.part_o[(pb + s + u) * p.R + c];
#pragma unroll
      for (int u = 0; u < 16; ++u) v += ws[s + u] * x[u];
    }
    for (; s < p.ns; ++s) v += ws[s] * p.part_o[(pb + s) * p.R + c];
    os[c] = v;
  }
  __syncthreads();
  T* O = static_cast<T*>(p.o) + (static_cast<int64_t>(b) * p.H + h) * p.vdim;
  float acc[U];
#pragma unroll
  for (int u = 0; u < U; ++u) acc[u] = 0.f;
  for (int c = lane * VEC; c < p.R; c += 64 * VEC) {
    if (c != lane * VEC) load_w(c);
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int e = 0; e < VEC; ++e) acc[u] += wv[u][e] * os[c + e];
  }
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const float s = wave_sum(acc[u]);
    if (lane == 0 && v0 + u < p.vdim) O[v0 + u] = from_f<T>(s);
  }
}

template <typename T>
void prepare(const void* down, int64_t ld, const void* qw, const void* kw, float eps, void* cq, void* latent,
             int64_t l_sb, int64_t l_st, const int64_t* slot, const int* kv_start, const float* cos_t,
             const float* sin_t, int B, int Tn, int qr, int R, int rot, int tcap, hipStream_t st) {
  const dim3 g(static_cast<unsigned>(B) * Tn);
  const bool vec = ld % 8 == 0 && qr % 8 == 0 && R % 8 == 0 && l_st % 8 == 0 && l_sb % 8 == 0 &&
                   (reinterpret_cast<uintptr_t>(down) | reinterpret_cast<uintptr_t>(qw) | reinterpret_cast<uintptr_t>(kw) |
                    reinterpret_cast<uintptr_t>(cq) | reinterpret_cast<uintptr_t>(latent)) % 16 == 0;
#define DLA_PREP(V)                                                                                                  \
  latent_prepare_kernel<T, V><<<g, 128, 0, st>>>(static_cast<const T*>(down), ld, static_cast<const T*>(qw),        \
                                                 static_cast<const T*>(kw), eps, static_cast<T*>(cq),               \
                                                 static_cast<T*>(latent), l_sb, l_st, slot, kv_start, cos_t, sin_t, \
                                                 Tn, qr, R, rot, tcap)
  if (vec) DLA_PREP(8);
  else DLA_PREP(1);
#undef DLA_PREP
}

template <typename T>
void attend_any(const LatentParams& p, int BN, hipStream_t st) {
  const int64_t lds = decode_lds<T>(p, BN);
  const dim3 gd(p.ns, (p.H + 15) / 16, p.B);
  const int nt = (p.R + 63) / 64;
#define DLA_DEC(NT)                                  \
  {                                                  \
    allow_lds(latent_decode_kernel<T, NT>, lds);     \
    latent_decode_kernel<T, NT><<<gd, 256, lds, st>>>(p, BN); \
  }
  if (nt <= 2) DLA_DEC(2)
  else if (nt <= 4) DLA_DEC(4)
  else if (nt <= 8) DLA_DEC(8)
  else DLA_DEC(16)
#undef DLA_DEC
}

template <typename T>
void decode(const LatentParams& p, int BN, hipStream_t st) {
  const bool vec = p.R % 8 == 0 && reinterpret_cast<uintptr_t>(p.kv_up) % 16 == 0;
  const dim3 ga(p.H, (p.R + 63) / 64);
  if (sizeof(T) == 2 && vec && p.dim % 8 == 0 && p.rot % 8 == 0 && p.dim <= 256 && reinterpret_cast<uintptr_t>(p.q) % 16 == 0) {
    if (p.dim <= 64) latent_absorb_mfma_kernel<2><<<ga, 256, 0, st>>>(p);
    else if (p.dim <= 128) latent_absorb_mfma_kernel<4><<<ga, 256, 0, st>>>(p);
    else latent_absorb_mfma_kernel<8><<<ga, 256, 0, st>>>(p);
  } else if (vec) latent_absorb_kernel<T, 8><<<ga, 256, 0, st>>>(p);
  else latent_absorb_kernel<T, 1><<<ga, 256, 0, st>>>(p);
  if (sizeof(T) == 2 && latent_decode_mfma_ok(p)) launch_latent_decode_mfma(p, st);
  else attend_any<T>(p, BN, st);
  const dim3 gc(p.H, p.B, (p.vdim + kCombV - 1) / kCombV);
  if (vec) latent_combine_kernel<T, 8><<<gc, 256, 4 * p.R, st>>>(p);
  else latent_combine_kernel<T, 1><<<gc, 256, 4 * p.R, st>>>(p);
}

}  // namespace

void launch_latent_prepare(bool bf16, const void* down, int64_t ld, const void* qw, const void* kw, float eps, void* cq,
                           void* latent, int64_t l_sb, int64_t l_st, const int64_t* slot, const int* kv_start,
                           const float* cos_t, const float* sin_t, int B, int Tn, int qr, int R, int rot, int tcap,
                           hipStream_t st) {
  if (bf16) prepare<bf16_t>(down, ld, qw, kw, eps, cq, latent, l_sb, l_st, slot, kv_start, cos_t, sin_t, B, Tn, qr, R, rot, tcap, st);
  else prepare<float>(down, ld, qw, kw, eps, cq, latent, l_sb, l_st, slot, kv_start, cos_t, sin_t, B, Tn, qr, R, rot, tcap, st);
}

// waves per workgroup of the any-size prefill kernel, 0 if the head sizes do not fit in LDS
int latent_prefill_waves(bool bf16, const LatentParams& p) {
  return bf16 ? prefill_waves<bf16_t>(p) : prefill_waves<float>(p);
}

void launch_latent_prefill_any(bool bf16, const LatentParams& p, hipStream_t st) {
  const int nw = latent_prefill_waves(bf16, p);
  const dim3 g((p.T + 16 * nw - 1) / (16 * nw), p.H, p.B);
  if (bf16) {
    allow_lds(latent_prefill_any_kernel<bf16_t>, prefill_lds<bf16_t>(p, nw));
    latent_prefill_any_kernel<bf16_t><<<g, 64 * nw, prefill_lds<bf16_t>(p, nw), st>>>(p);
  } else {
    allow_lds(latent_prefill_any_kernel<float>, prefill_lds<float>(p, nw));
    latent_prefill_any_kernel<float><<<g, 64 * nw, prefill_lds<float>(p, nw), st>>>(p);
  }
}

// keys per tile of the decode kernel, 0 if the latent does not fit in LDS
int latent_decode_tile(bool bf16, const LatentParams& p) {
  if (p.R > 1024) return 0;
  for (int bn = 64; bn >= 32; bn /= 2)
    if ((bf16 ? decode_lds<bf16_t>(p, bn) : decode_lds<float>(p, bn)) <= kLdsMax) return bn;
  return 0;
}

void launch_latent_decode(bool bf16, const LatentParams& p, int tile, hipStream_t st) {
  if (bf16) decode<bf16_t>(p, tile, st);
  else decode<float>(p, tile, st);
}

}  // namespace dla
