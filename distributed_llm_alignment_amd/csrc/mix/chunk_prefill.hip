// Attention inside chunks, prompts, on bf16 MFMA 32x32x16 (head sizes up to 256; other sizes and fp32:
// chunk_attn.hip).
//
// A workgroup is 4 waves x 32 queries of one (sequence, head); key tiles of 64. Scores are formed
// transposed, S^T = K Q^T, so a lane owns one query's column (softmax is in-lane plus one xor-32 step)
// and the exponentiated accumulator is the PV operand as it stands; V^T comes out of the row image by
// transposed LDS reads. The weights go into the PV product as hi + lo bf16 planes (mma.h). Keys are
// addressed by position: the portion's own, and before them the cached ones of the chunk it starts in.
// A query's first visible position is a per-lane value, so only the tiles that a chunk's edge or the
// diagonal cuts are masked. Heads are the fastest grid dimension, the longest query blocks start first.
#include "mix_params.h"
#include "mma.h"

namespace dla {
namespace {

constexpr float kLog2e = 1.4426950408889634f;
constexpr int kBM = 128, kBN = 64, kThreads = 256;
typedef __attribute__((address_space(3))) s16x4 lds_s16x4;

// LDS row strides (elements). K rows are read 16 B per lane along rows: stride an odd multiple of
// 16 B. V rows are read transposed, 4 rows x 64 B per half wave: stride an odd multiple of 64 B.
__host__ __device__ constexpr int k_stride(int nk) { return 16 * nk + 8; }
__host__ __device__ constexpr int v_stride(int nv) { return 32 * nv + (nv % 2 ? 0 : 32); }

__device__ __forceinline__ f32x16 mfma32(s16x8 a, s16x8 b, f32x16 c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0);
}

// NK: 16-wide score steps (16 NK >= dim), NV: 32-wide value tiles (32 NV >= vdim)
template <int NK, int NV>
__global__ __launch_bounds__(kThreads, NK > 8 || NV > 4 ? 1 : 2) void chunk_prefill_kernel(ChunkAttnParams p, int nqb) {
  constexpr int SK = k_stride(NK), SV = v_stride(NV);
  constexpr int CK = 2 * NK, CV = 4 * NV;                        // 16-byte chunks per row
  constexpr int LK = kBN * CK / kThreads, LV = kBN * CV / kThreads;  // chunks per thread
  static_assert(kBN * CK % kThreads == 0 && kBN * CV % kThreads == 0, "staging geometry");
  __shared__ __attribute__((aligned(16))) bf16_t ks[kBN * SK];
  __shared__ __attribute__((aligned(16))) bf16_t vs[kBN * SV];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, c32 = lane & 31, g = lane >> 5;
  const int h = blockIdx.x % p.H, b = (blockIdx.x / p.H) % p.B, qb = nqb - 1 - blockIdx.x / (p.H * p.B);
  const int q0 = qb * kBM, hk = h / (p.H / p.G);
  const int off = static_cast<int>(p.base) - (p.kv_start ? p.kv_start[b] : 0);  // position of query 0 (< 0: padding)
  const int64_t kst = static_cast<int64_t>(p.G) * p.dim, vst = static_cast<int64_t>(p.G) * p.vdim;
  const bf16_t* K = static_cast<const bf16_t*>(p.k) + static_cast<int64_t>(b) * p.T * kst + hk * p.dim;
  const bf16_t* V = static_cast<const bf16_t*>(p.v) + static_cast<int64_t>(b) * p.T * vst + hk * p.vdim;
  const int64_t cb = (static_cast<int64_t>(b) * p.G + hk) * p.rows;
  const int cfirst = off > 0 ? off - off % p.chunk : 0;  // position of cache row 0
  const bf16_t* KC = static_cast<const bf16_t*>(p.kc) + cb * p.dim;
  const bf16_t* VC = static_cast<const bf16_t*>(p.vc) + cb * p.vdim;

  // this lane's query (B operand: column c32, k = 16 s + 8 g ..)
  const int tq = q0 + wave * 32 + c32, qpos = off + tq;
  const int qlo = qpos > 0 ? qpos - qpos % p.chunk : 0;
  s16x8 qf[NK];
  {
    const bf16_t* row = static_cast<const bf16_t*>(p.q) + ((static_cast<int64_t>(b) * p.T + min(tq, p.T - 1)) * p.H + h) * p.dim;
#pragma unroll
    for (int s = 0; s < NK; ++s) {
      const int d = 16 * s + 8 * g;
      bf16x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
      if (d < p.dim) v = load_bf16x8(row + d);
      qf[s] = __builtin_bit_cast(s16x8, v);
    }
  }

  const int first = max(off + q0, 0), lo = first - first % p.chunk, hi = off + min(q0 + kBM, p.T);
  // the wave's own query positions [wlo, whi] and the first positions their chunks start at
  const int wlo = off + q0 + wave * 32, whi = wlo + 31;
  const int wfirst = wlo > 0 ? wlo - wlo % p.chunk : 0, wlast = whi > 0 ? whi - whi % p.chunk : 0;
  const float c = p.scale * kLog2e;
  float m_run = -INFINITY, l_run = 0.f;
  f32x16 o[NV];
#pragma unroll
  for (int t = 0; t < NV; ++t)
#pragma unroll
    for (int i = 0; i < 16; ++i) o[t][i] = 0.f;

  bf16x8 kreg[LK], vreg[LV];
  auto load_tile = [&](int c0) {
#pragma unroll
    for (int j = 0; j < LK; ++j) {
      const int i = threadIdx.x + kThreads * j, n = i / CK, d = (i % CK) * 8;
      const int s = min(c0 + n, hi - 1);  // rows past the end repeat the last one (masked)
      bf16x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
      if (d < p.dim) v = load_bf16x8((s >= off ? K + (s - off) * kst : KC + static_cast<int64_t>(s - cfirst) * p.dim) + d);
      kreg[j] = v;
    }
#pragma unroll
    for (int j = 0; j < LV; ++j) {
      const int i = threadIdx.x + kThreads * j, n = i / CV, d = (i % CV) * 8;
      const int s = min(c0 + n, hi - 1);
      bf16x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
      if (d < p.vdim) v = load_bf16x8((s >= off ? V + (s - off) * vst : VC + static_cast<int64_t>(s - cfirst) * p.vdim) + d);
      vreg[j] = v;
    }
  };
  if (lo < hi) load_tile(lo);
  for (int c0 = lo; c0 < hi; c0 += kBN) {
    __syncthreads();  // every wave is done with the last tile
#pragma unroll
    for (int j = 0; j < LK; ++j) {
      const int i = threadIdx.x + kThreads * j;
      store_bf16x8(ks + (i / CK) * SK + (i % CK) * 8, kreg[j]);
    }
#pragma unroll
    for (int j = 0; j < LV; ++j) {
      const int i = threadIdx.x + kThreads * j;
      store_bf16x8(vs + (i / CV) * SV + (i % CV) * 8, vreg[j]);
    }
    __syncthreads();
    if (c0 + kBN < hi) load_tile(c0 + kBN);
    if (c0 > whi || c0 + kBN <= wfirst) continue;  // nothing of this tile is visible to the wave's queries

    f32x16 s[2];
#pragma unroll
    for (int n = 0; n < 2; ++n) {
#pragma unroll
      for (int i = 0; i < 16; ++i) s[n][i] = 0.f;
      const bf16_t* kp = ks + (32 * n + c32) * SK + 8 * g;
#pragma unroll
      for (int k = 0; k < NK; ++k) s[n] = mfma32(__builtin_bit_cast(s16x8, load_bf16x8(kp + 16 * k)), qf[k], s[n]);
    }
    const bool whole = c0 + kBN - 1 <= wlo && c0 >= wlast && c0 + kBN <= hi;
    float mx = -INFINITY;
#pragma unroll
    for (int n = 0; n < 2; ++n)
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        float x = s[n][i] * c;
        if (!whole) {
          const int j = c0 + 32 * n + 8 * (i >> 2) + 4 * g + (i & 3);
          if (!(j < hi && j <= qpos && j >= qlo)) x = -INFINITY;
        }
        s[n][i] = x;
        mx = fmaxf(mx, x);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    if (__builtin_amdgcn_ballot_w64(mx > m_run)) {
      const float mn = fmaxf(m_run, mx);
      const float a = mn == -INFINITY ? 1.f : __builtin_amdgcn_exp2f(m_run - mn);
      m_run = mn;
      l_run *= a;
#pragma unroll
      for (int t = 0; t < NV; ++t)
#pragma unroll
        for (int i = 0; i < 16; ++i) o[t][i] *= a;
    }
    const float mu = m_run == -INFINITY ? 0.f : m_run;
    float l = 0.f;
#pragma unroll
    for (int n = 0; n < 2; ++n)
#pragma unroll
      for (int kb = 0; kb < 2; ++kb) {
        // 16 keys: slots e < 4 are keys 4g + e, e >= 4 keys 8 + 4g + e - 4 of this block of 16
        float pv[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          pv[e] = __builtin_amdgcn_exp2f(s[n][8 * kb + e] - mu);
          l += pv[e];
        }
        s16x8 ph, pl;
        Mma<bf16_t>::split(pv, ph, pl);
        const int r0 = 32 * n + 16 * kb + 4 * g;
        const bf16_t* vp = vs + (r0 + ((lane & 15) >> 2)) * SV + 16 * ((lane >> 4) & 1) + 4 * (lane & 3);
#pragma unroll
        for (int t = 0; t < NV; ++t) {
          const s16x4 v0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)(vp + 32 * t));
          const s16x4 v1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)(vp + 8 * SV + 32 * t));
          const s16x8 va = {v0[0], v0[1], v0[2], v0[3], v1[0], v1[1], v1[2], v1[3]};
          o[t] = mfma32(va, ph, o[t]);
          o[t] = mfma32(va, pl, o[t]);
        }
      }
    l_run += l;
  }
  l_run += __shfl_xor(l_run, 32, 64);
  if (tq >= p.T) return;
  const float inv = l_run > 0.f ? 1.f / l_run : 0.f;
  bf16_t* O = static_cast<bf16_t*>(p.o) + ((static_cast<int64_t>(b) * p.T + tq) * p.H + h) * p.vdim;
#pragma unroll
  for (int t = 0; t < NV; ++t)
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int v = 32 * t + 8 * u + 4 * g;
      if (v < p.vdim) {
        typedef uint32_t u32x2 __attribute__((ext_vector_type(2)));
        *reinterpret_cast<u32x2*>(O + v) = u32x2{pack2bf(o[t][4 * u] * inv, o[t][4 * u + 1] * inv),
                                                 pack2bf(o[t][4 * u + 2] * inv, o[t][4 * u + 3] * inv)};
      }
    }
}

template <int NK, int NV>
void go(const ChunkAttnParams& p, hipStream_t st) {
  const int nqb = (p.T + kBM - 1) / kBM;
  chunk_prefill_kernel<NK, NV><<<dim3(nqb * p.H * p.B), kThreads, 0, st>>>(p, nqb);
}

template <int NK>
void go_v(const ChunkAttnParams& p, hipStream_t st) {
  if (p.vdim <= 64) go<NK, 2>(p, st);
  else if (p.vdim <= 128) go<NK, 4>(p, st);
  else go<NK, 8>(p, st);
}

}  // namespace

bool chunk_prefill_mfma_ok(const ChunkAttnParams& p) {
  const auto al = [](const void* x) { return reinterpret_cast<uintptr_t>(x) % 16 == 0; };
  return p.dim % 8 == 0 && p.vdim % 8 == 0 && p.dim <= 256 && p.vdim <= 256 && al(p.q) && al(p.k) && al(p.v) && al(p.kc) &&
         al(p.vc) && al(p.o) && p.base + p.T < (1ll << 30) &&
         static_cast<int64_t>((p.T + kBM - 1) / kBM) * p.H * p.B < (1ll << 31);
}

void launch_chunk_prefill_mfma(const ChunkAttnParams& p, hipStream_t st) {
  const int nk = (p.dim + 15) / 16;
  if (nk <= 4) go_v<4>(p, st);
  else if (nk <= 8) go_v<8>(p, st);
  else go_v<16>(p, st);
}

}  // namespace dla
