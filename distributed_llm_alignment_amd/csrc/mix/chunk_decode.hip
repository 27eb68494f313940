// Attention inside chunks, one new token, on bf16 MFMA 16x16x32 (head sizes up to 256; other sizes and
// fp32: chunk_attn.hip).
//
// Workgroup = (key split, key head and up to 16 of its query heads, sequence), 4 waves; a wave takes 32
// keys at a time and keeps its own running softmax; the waves merge once at the end. S^T = K q^T reads
// the key rows as they lie; the exponentiated accumulator is the A operand of the PV product as it
// stands (fp32 weights, hi + lo planes), the value rows go through a wave-private LDS image and come
// back transposed. Rows 0 .. pos % chunk of the cache are what the token sees: no masks but the end.
#include "mix_params.h"
#include "mma.h"

namespace dla {
namespace {

constexpr float kLog2e = 1.4426950408889634f;
constexpr int kBN = 128;  // keys per workgroup and step
typedef __attribute__((address_space(3))) s16x4 lds_s16x4;
__device__ __forceinline__ s16x4 tr4(const bf16_t* p) { return __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)(p)); }

// NK: 32-wide steps over dim, NV: 16-wide value tiles
template <int NK, int NV>
__global__ __launch_bounds__(256) void chunk_decode_kernel(ChunkAttnParams p) {
  constexpr int SV = 16 * NV + 16, CV = 2 * NV;           // value row stride, 16-byte pieces per row
  constexpr int LV = 32 * CV / 64;                        // pieces per lane
  constexpr int kImg = 4 * 32 * SV * 2, kAcc = 4 * 16 * (16 * NV) * 4;
  __shared__ __attribute__((aligned(16))) unsigned char smem[kImg > kAcc ? kImg : kAcc];
  __shared__ float ml[4][16][2];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane & 15, g = lane >> 4;
  const int grp = p.H / p.G, ng = (grp + 15) / 16;
  const int hk = blockIdx.y / ng, h0 = hk * grp + (blockIdx.y % ng) * 16, b = blockIdx.z, split = blockIdx.x;
  const int nh = min(16, (hk + 1) * grp - h0);
  bf16_t* img = reinterpret_cast<bf16_t*>(smem) + wave * 32 * SV;
  const int64_t pos = max(p.slot[0] - (p.kv_start ? p.kv_start[b] : 0), static_cast<int64_t>(0));
  const int n = static_cast<int>(min(pos % p.chunk + 1, static_cast<int64_t>(p.rows)));
  const int per = ((n + p.ns - 1) / p.ns + 31) / 32 * 32, k0 = split * per, k1 = min(k0 + per, n);
  const int64_t cb = (static_cast<int64_t>(b) * p.G + hk) * p.rows;
  const bf16_t* K = static_cast<const bf16_t*>(p.kc) + cb * p.dim;
  const bf16_t* V = static_cast<const bf16_t*>(p.vc) + cb * p.vdim;
  s16x8 qf[NK];
  {
    const bf16_t* q = static_cast<const bf16_t*>(p.q) + (static_cast<int64_t>(b) * p.H + h0 + min(r, nh - 1)) * p.dim;
#pragma unroll
    for (int k = 0; k < NK; ++k) {
      const int d = 32 * k + 8 * g;
      bf16x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
      if (d < p.dim) v = load_bf16x8(q + d);
      qf[k] = __builtin_bit_cast(s16x8, v);
    }
  }
  f32x4 acc[NV];
#pragma unroll
  for (int t = 0; t < NV; ++t) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m_run = -INFINITY, l_run = 0.f;  // of head r
  const float c = p.scale * kLog2e;
  for (int c0 = k0 + 32 * wave; c0 < k1; c0 += kBN) {
    s16x8 kf[2][NK];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      const bf16_t* row = K + static_cast<int64_t>(min(c0 + 16 * t + r, k1 - 1)) * p.dim;
#pragma unroll
      for (int k = 0; k < NK; ++k) {
        const int d = 32 * k + 8 * g;
        bf16x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
        if (d < p.dim) v = load_bf16x8(row + d);
        kf[t][k] = __builtin_bit_cast(s16x8, v);
      }
    }
    bf16x8 vreg[LV];
#pragma unroll
    for (int j = 0; j < LV; ++j) {
      const int i = lane + 64 * j, s = i / CV, d = (i % CV) * 8;
      bf16x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
      if (d < p.vdim) v = load_bf16x8(V + static_cast<int64_t>(min(c0 + s, k1 - 1)) * p.vdim + d);
      vreg[j] = v;
    }
    // S^T: this lane holds keys c0 + 16 t + 4 g + i of head r
    f32x4 s[2];
    float mx = -INFINITY;
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      s[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < NK; ++k) s[t] = Mma<bf16_t>::mma(kf[t][k], qf[k], s[t]);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        s[t][i] = c0 + 16 * t + 4 * g + i < k1 ? s[t][i] * c : -INFINITY;
        mx = fmaxf(mx, s[t][i]);
      }
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));  // (key c0 is there: finite)
    if (__builtin_amdgcn_ballot_w64(mx > m_run)) {
      const float mn = fmaxf(m_run, mx), a = __builtin_amdgcn_exp2f(m_run - mn);
      m_run = mn;
      l_run *= a;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float ai = __shfl(a, 4 * g + i, 64);
#pragma unroll
        for (int t = 0; t < NV; ++t) acc[t][i] *= ai;
      }
    }
    float pv[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      pv[e] = __builtin_amdgcn_exp2f(s[e >> 2][e & 3] - m_run);
      l_run += pv[e];
    }
    s16x8 ph, pl;
    Mma<bf16_t>::split(pv, ph, pl);
    __builtin_amdgcn_wave_barrier();  // (the image is this wave's own: its LDS accesses stay in order)
#pragma unroll
    for (int j = 0; j < LV; ++j) {
      const int i = lane + 64 * j;
      store_bf16x8(img + (i / CV) * SV + (i % CV) * 8, vreg[j]);
    }
    __builtin_amdgcn_wave_barrier();
    const bf16_t* vp = img + (4 * g + (r >> 2)) * SV + 4 * (r & 3);
#pragma unroll
    for (int t = 0; t < NV; ++t) {
      const s16x4 v0 = tr4(vp + 16 * t), v1 = tr4(vp + 16 * SV + 16 * t);
      const s16x8 bv = {v0[0], v0[1], v0[2], v0[3], v1[0], v1[1], v1[2], v1[3]};
      acc[t] = Mma<bf16_t>::mma(ph, bv, acc[t]);
      acc[t] = Mma<bf16_t>::mma(pl, bv, acc[t]);
    }
  }
  l_run += __shfl_xor(l_run, 16, 64);
  l_run += __shfl_xor(l_run, 32, 64);
  if (g == 0) {
    ml[wave][r][0] = m_run;
    ml[wave][r][1] = l_run;
  }
  __syncthreads();  // every wave is done with its image
  float* os = reinterpret_cast<float*>(smem);
#pragma unroll
  for (int t = 0; t < NV; ++t)
#pragma unroll
    for (int i = 0; i < 4; ++i) os[(wave * 16 + 4 * g + i) * (16 * NV) + 16 * t + r] = acc[t][i];
  __syncthreads();
  for (int i = threadIdx.x; i < nh * p.vdim; i += 256) {
    const int hh = i / p.vdim, v = i % p.vdim;
    const float m = fmaxf(fmaxf(ml[0][hh][0], ml[1][hh][0]), fmaxf(ml[2][hh][0], ml[3][hh][0]));
    float o = 0.f, l = 0.f;
    if (m != -INFINITY) {
#pragma unroll
      for (int w = 0; w < 4; ++w) {
        const float e = exp2f(ml[w][hh][0] - m);
        o += e * os[(w * 16 + hh) * (16 * NV) + v];
        l += e * ml[w][hh][1];
      }
    }
    const int64_t bh = static_cast<int64_t>(b) * p.H + h0 + hh;
    if (p.ns == 1) {
      static_cast<bf16_t*>(p.o)[bh * p.vdim + v] = f2bf(o / l);
    } else {
      p.part_o[(bh * p.ns + split) * p.vdim + v] = o;
      if (v == 0) {
        p.part_ml[2 * (bh * p.ns + split)] = m;
        p.part_ml[2 * (bh * p.ns + split) + 1] = l;
      }
    }
  }
}

template <int NK, int NV>
void go(const ChunkAttnParams& p, hipStream_t st) {
  const int grp = p.H / p.G;
  chunk_decode_kernel<NK, NV><<<dim3(p.ns, p.G * ((grp + 15) / 16), p.B), 256, 0, st>>>(p);
}

template <int NK>
void go_v(const ChunkAttnParams& p, hipStream_t st) {
  if (p.vdim <= 64) go<NK, 4>(p, st);
  else if (p.vdim <= 128) go<NK, 8>(p, st);
  else go<NK, 16>(p, st);
}

}  // namespace

bool chunk_decode_mfma_ok(const ChunkAttnParams& p) {
  const auto al = [](const void* x) { return reinterpret_cast<uintptr_t>(x) % 16 == 0; };
  return p.dim % 8 == 0 && p.vdim % 8 == 0 && p.dim <= 256 && p.vdim <= 256 && p.rows < (1 << 30) && al(p.q) && al(p.kc) &&
         al(p.vc);
}

void launch_chunk_decode_mfma(const ChunkAttnParams& p, hipStream_t st) {
  if (p.dim <= 64) go_v<2>(p, st);
  else if (p.dim <= 128) go_v<4>(p, st);
  else go_v<8>(p, st);
}

}  // namespace dla
