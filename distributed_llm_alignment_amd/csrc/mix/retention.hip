// Retention (linear attention with one fixed decay per head, no denominator) for gfx950.
//
//   S_t = decay S_(t-1) + k_t v_t^T,  o_t = S_t^T q_t,  y = o / rms(o) * silu(g)
//
// Prompt portions run in chunks of C tokens, three launches:
//   state   every chunk's own contribution K'^T V with k'_t = k_t decay^(len-1-t)      (B H nc WGs)
//   scan    start state of every chunk: S <- decay^len S + contribution                (B H dim vdim threads)
//   output  (Q K^T o decay^(t-s)) V + decay^(t+1) Q S_start, per-head norm, gate       (B H nc WGs)
// Decode (and portions shorter than a chunk is worth, and head sizes whose tiles do not fit in LDS)
// runs the recurrence itself: one workgroup per (sequence, head), one read-modify-write of the state
// per token.
//
// The state is kept transposed, [vdim, dim]: a row is what one output column needs, contiguous.
// Rotated keys, decayed scores and the state are fp32 values; on bf16 MFMAs they travel as hi + lo
// planes (mma.h). q, k and v come out of the projections in the compute dtype.
#include "mix_params.h"
#include "mma.h"

namespace dla {

bool retention_mfma_ok(const RetentionParams&);  // retention_mfma.hip
void launch_retention_state_mfma(const RetentionParams&, hipStream_t);
void launch_retention_output_mfma(const RetentionParams&, hipStream_t);

namespace {

template <typename T>
constexpr int pad16() { return 16 / static_cast<int>(sizeof(T)); }  // row pad of an LDS tile (16 bytes)

struct RetHead {  // one (batch, head)'s rows
  int b, h, kv0;
  float l2;
};

// stage rows [t0, t0 + len) of the rotated q or k (scaled), zero beyond len / in padding, as planes
// [C][ldr] (TRANS: [dim][ldr])
template <typename T, int VEC, bool TRANS>
__device__ __forceinline__ void stage_rotated(const RetentionParams& p, const RetHead& hd, int off, int t0, int len, int C,
                                              int dp, T* dst, int ldr, int plane, float scale, bool is_key, bool decayed) {
  const int nv = dp / VEC;
  const int half = p.rot >> 1;
  for (int i = threadIdx.x; i < C * nv; i += blockDim.x) {
    const int t = TRANS ? i % C : i / nv, i0 = (TRANS ? i / C : i % nv) * VEC;
    float v[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = 0.f;
    const int64_t pos = p.base + t0 + t - hd.kv0;
    if (t < len && i0 < p.dim && (pos >= 0 || !is_key)) {
      const T* row = static_cast<const T*>(p.qkvg) + (static_cast<int64_t>(hd.b) * p.T + t0 + t) * p.ld + off;
      const int64_t pp = pos < 0 ? 0 : pos;
      load_rotated<T, VEC>(row, i0, p.rot, p.cos_t + pp * half, p.sin_t + pp * half, v);
      const float f = decayed ? scale * exp2f(static_cast<float>(len - 1 - t) * hd.l2) : scale;
#pragma unroll
      for (int e = 0; e < VEC; ++e) v[e] *= f;
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) put_planes<T>(TRANS ? dst + (i0 + e) * ldr + t : dst + t * ldr + i0 + e, plane, v[e]);
  }
}

// V rows transposed: vt[v][t], zero beyond len / vdim and in padding (0 x whatever a padding row holds)
template <typename T, int VEC>
__device__ __forceinline__ void stage_vt(const RetentionParams& p, const RetHead& hd, int off, int t0, int len, int C,
                                         int vp, T* vt, int ldv) {
  const int nv = vp / VEC;
  for (int i = threadIdx.x; i < C * nv; i += blockDim.x) {
    const int t = i % C, i0 = (i / C) * VEC;
    float v[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = 0.f;
    if (t < len && i0 < p.vdim && p.base + t0 + t >= hd.kv0)
      load_vec<T, VEC>(static_cast<const T*>(p.qkvg) + (static_cast<int64_t>(hd.b) * p.T + t0 + t) * p.ld + off + i0, v);
#pragma unroll
    for (int e = 0; e < VEC; ++e) vt[(i0 + e) * ldv + t] = from_f<T>(v[e]);
  }
}

__device__ __forceinline__ RetHead ret_head(const RetentionParams& p, int h, int b) {
  return RetHead{b, h, p.kv_start ? p.kv_start[b] : 0, p.decay[p.H + h]};
}

// grid (nc, H, B), 256 threads
template <typename T, int VEC>
__global__ __launch_bounds__(256) void ret_state_kernel(RetentionParams p) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  using M = Mma<T>;
  const RetHead hd = ret_head(p, blockIdx.y, blockIdx.z);
  const int C = p.chunk, t0 = blockIdx.x * C, len = min(C, p.T - t0);
  const int dp = round_up(p.dim, 32), vp = round_up(p.vdim, 16), ldr = C + pad16<T>();
  T* kt = reinterpret_cast<T*>(smem);
  T* vt = kt + M::PL * dp * ldr;
  const int Hd = p.H * p.dim;
  stage_rotated<T, VEC, true>(p, hd, Hd + hd.h * p.dim, t0, len, C, dp, kt, ldr, dp * ldr, p.kscale, true, true);
  stage_vt<T, VEC>(p, hd, 2 * Hd + hd.h * p.vdim, t0, len, C, vp, vt, ldr);
  __syncthreads();
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane & 15, g = lane >> 4;
  float* W = p.work + ((static_cast<int64_t>(hd.b) * p.H + hd.h) * p.nc + blockIdx.x) * p.vdim * p.dim;
  const int ndt = (p.dim + 15) / 16;
  for (int tile = wave; tile < (vp / 16) * ndt; tile += 4) {
    const int v0 = tile / ndt * 16, d0 = tile % ndt * 16;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    for (int k = 0; k < C; k += M::KS) {
      const auto a = M::row(vt + (v0 + r) * ldr + k + g * M::KV);
      const T* kp = kt + (d0 + r) * ldr + k + g * M::KV;
      acc = M::mma(a, M::row(kp), acc);
      if constexpr (M::PL == 2) acc = M::mma(a, M::row(kp + dp * ldr), acc);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int v = v0 + 4 * g + i, d = d0 + r;
      if (v < p.vdim && d < p.dim) W[static_cast<int64_t>(v) * p.dim + d] = acc[i];
    }
  }
}

// grid (ceil(vdim dim / VEC / 256), H, B): work[c] <- start state of chunk c; state <- final state
template <int VEC>
__global__ __launch_bounds__(256) void ret_scan_kernel(RetentionParams p) {
  const int64_t n = static_cast<int64_t>(p.vdim) * p.dim;
  const int64_t i = (blockIdx.x * 256ll + threadIdx.x) * VEC;
  if (i >= n) return;
  const int64_t bh = static_cast<int64_t>(blockIdx.z) * p.H + blockIdx.y;
  const float l2 = p.decay[p.H + blockIdx.y];
  float* st = p.state + bh * n + i;
  float* W = p.work + bh * p.nc * n + i;
  float s[VEC];
#pragma unroll
  for (int e = 0; e < VEC; ++e) s[e] = 0.f;
  if (!p.fresh) load_vec<float, VEC>(st, s);
  const float full = exp2f(static_cast<float>(p.chunk) * l2);
  constexpr int U = 8;
  for (int c0 = 0; c0 < p.nc; c0 += U) {
    float w[U][VEC];
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (c0 + u < p.nc) load_vec<float, VEC>(W + (c0 + u) * n, w[u]);
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = c0 + u;
      if (c >= p.nc) break;
      store_vec<float, VEC>(W + c * n, s);
      const float f = c == p.nc - 1 ? exp2f(static_cast<float>(p.T - c * p.chunk) * l2) : full;
#pragma unroll
      for (int e = 0; e < VEC; ++e) s[e] = f * s[e] + w[u][e];
    }
  }
  store_vec<float, VEC>(st, s);
}

__host__ __device__ inline int ret_k_elems(int C, int dp, int pl, int pad) {
  const int k = pl * C * (dp + pad), pq = pl * C * (C + pad);
  return k > pq ? k : pq;  // the scores overlay the keys
}

// grid (nc, H, B), 256 threads; CT = C / 16
template <typename T, int VEC, int CT>
__global__ __launch_bounds__(256) void ret_output_kernel(RetentionParams p) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  using M = Mma<T>;
  constexpr int C = 16 * CT, NP = CT * CT / 4;  // score tiles per wave
  const RetHead hd = ret_head(p, blockIdx.y, blockIdx.z);
  const int t0 = blockIdx.x * C, len = min(C, p.T - t0);
  const int dp = round_up(p.dim, 32), vp = round_up(p.vdim, 16);
  const int ldd = dp + pad16<T>(), ldc = C + pad16<T>(), ldo = vp + 4;
  T* qs = reinterpret_cast<T*>(smem);
  T* ks = qs + M::PL * C * ldd;
  T* vt = ks + ret_k_elems(C, dp, M::PL, pad16<T>());
  float* os = reinterpret_cast<float*>(vt + vp * ldc);
  T* ps = ks;
  const int Hd = p.H * p.dim, Hv = p.H * p.vdim;
  stage_rotated<T, VEC, false>(p, hd, hd.h * p.dim, t0, len, C, dp, qs, ldd, C * ldd, 1.f, false, false);
  stage_rotated<T, VEC, false>(p, hd, Hd + hd.h * p.dim, t0, len, C, dp, ks, ldd, C * ldd, p.kscale, true, false);
  stage_vt<T, VEC>(p, hd, 2 * Hd + hd.h * p.vdim, t0, len, C, vp, vt, ldc);
  __syncthreads();
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane & 15, g = lane >> 4;

  f32x4 sc[NP];
#pragma unroll
  for (int j = 0; j < NP; ++j) {
    const int rt = (wave + 4 * j) / CT, ct = (wave + 4 * j) % CT;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    if (ct <= rt) {
      for (int k = 0; k < dp; k += M::KS) {
        const T* qp = qs + (rt * 16 + r) * ldd + k + g * M::KV;
        const T* kp = ks + (ct * 16 + r) * ldd + k + g * M::KV;
        const auto a = M::row(qp), b = M::row(kp);
        acc = M::mma(a, b, acc);
        if constexpr (M::PL == 2) {
          acc = M::mma(M::row(qp + C * ldd), b, acc);
          acc = M::mma(a, M::row(kp + C * ldd), acc);
        }
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int dt = (rt * 16 + 4 * g + i) - (ct * 16 + r);
        acc[i] = dt >= 0 ? acc[i] * exp2f(static_cast<float>(dt) * hd.l2) : 0.f;
      }
    }
    sc[j] = acc;
  }
  __syncthreads();  // every wave is done with the keys
#pragma unroll
  for (int j = 0; j < NP; ++j) {
    const int rt = (wave + 4 * j) / CT, ct = (wave + 4 * j) % CT;
#pragma unroll
    for (int i = 0; i < 4; ++i) put_planes<T>(ps + (rt * 16 + 4 * g + i) * ldc + ct * 16 + r, C * ldc, sc[j][i]);
  }
  __syncthreads();

  const float* S = p.work + ((static_cast<int64_t>(hd.b) * p.H + hd.h) * p.nc + blockIdx.x) * p.vdim * p.dim;
  const bool carried = !p.fresh || blockIdx.x > 0;  // chunk 0 of a fresh sequence starts at zero
  for (int v0 = wave * 16; v0 < vp; v0 += 64) {
    f32x4 acc[CT], acs[CT];
#pragma unroll
    for (int t = 0; t < CT; ++t) acc[t] = acs[t] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int k = 0; k < C; k += M::KS) {
      const auto b = M::row(vt + (v0 + r) * ldc + k + g * M::KV);
#pragma unroll
      for (int t = 0; t < CT; ++t) {
        if (k > t * 16 + 15) continue;  // scores above the diagonal are zero
        const T* pp = ps + (t * 16 + r) * ldc + k + g * M::KV;
        acc[t] = M::mma(M::row(pp), b, acc[t]);
        if constexpr (M::PL == 2) acc[t] = M::mma(M::row(pp + C * ldc), b, acc[t]);
      }
    }
    if (carried) {
      const float* srow = S + static_cast<int64_t>(v0 + r) * p.dim;
      for (int k = 0; k < dp; k += M::KS) {
        float sv[8];
        const int kk = k + g * M::KV;
#pragma unroll
        for (int e = 0; e < M::KV; ++e) sv[e] = 0.f;
        if (v0 + r < p.vdim) {
          if constexpr (VEC == 8) {
            if (kk < p.dim) load_vec<float, M::KV>(srow + kk, sv);
          } else {
#pragma unroll
            for (int e = 0; e < M::KV; ++e)
              if (kk + e < p.dim) sv[e] = srow[kk + e];
          }
        }
        typename M::Frag bh, bl;
        M::split(sv, bh, bl);
#pragma unroll
        for (int t = 0; t < CT; ++t) {
          const T* qp = qs + (t * 16 + r) * ldd + kk;
          const auto a = M::row(qp);
          acs[t] = M::mma(a, bh, acs[t]);
          if constexpr (M::PL == 2) {
            acs[t] = M::mma(M::row(qp + C * ldd), bh, acs[t]);
            acs[t] = M::mma(a, bl, acs[t]);
          }
        }
      }
    }
#pragma unroll
    for (int t = 0; t < CT; ++t)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int m = t * 16 + 4 * g + i;
        os[m * ldo + v0 + r] = acc[t][i] + acs[t][i] * exp2f(static_cast<float>(m + 1) * hd.l2);
      }
  }
  __syncthreads();
  for (int t = wave; t < len; t += 4) {
    float ss = 0.f;
    for (int v = lane; v < p.vdim; v += 64) ss += os[t * ldo + v] * os[t * ldo + v];
    const float rs = rsqrtf(wave_sum(ss) / p.vdim + p.eps);
    const int64_t row = static_cast<int64_t>(hd.b) * p.T + t0 + t;
    const T* gr = static_cast<const T*>(p.qkvg) + row * p.ld + 2 * Hd + Hv + hd.h * p.vdim;
    T* yr = static_cast<T*>(p.y) + row * Hv + hd.h * p.vdim;
    for (int v = lane; v < p.vdim; v += 64) {
      const float gv = to_f<T>(gr[v]);
      yr[v] = from_f<T>(os[t * ldo + v] * rs * (gv / (1.f + expf(-gv))));
    }
  }
}

// The recurrence, token by token. grid (H, B, vsplit), NT threads; vsplit > 1 (decode of few rows): each
// workgroup owns a range of the value rows and publishes its outputs with write-through stores; the
// last to arrive at the (sequence, head) counter re-arms it, acquires once and does the norm and
// gate. Nobody waits for anybody. a row of the state (one v) belongs to a
// group of `lpr` lanes, each lane to VEC-element pieces of it.
constexpr int kRecThreads = 512;
template <typename T, int VEC>
__global__ __launch_bounds__(kRecThreads) void ret_recurrent_kernel(RetentionParams p, int lpr) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  __shared__ float scratch[kRecThreads / 64];
  float* qs = reinterpret_cast<float*>(smem);
  float* ks = qs + round_up(p.dim, 4);
  float* vs = ks + round_up(p.dim, 4);
  float* os = vs + p.vdim;
  const RetHead hd = ret_head(p, blockIdx.x, blockIdx.y);
  const int64_t base = p.slot ? p.slot[0] : p.base;
  const float dec = p.decay[hd.h];
  const int Hd = p.H * p.dim, Hv = p.H * p.vdim, half = p.rot >> 1;
  float* S = p.state + (static_cast<int64_t>(hd.b) * p.H + hd.h) * p.vdim * p.dim;
  const int grp = threadIdx.x / lpr, li = threadIdx.x % lpr, ngrp = kRecThreads / lpr;
  constexpr int U = 8;
  const int per = (p.vdim + p.vsplit - 1) / p.vsplit, vlo = blockIdx.z * per, vhi = min(vlo + per, p.vdim);
  for (int t = 0; t < p.T; ++t) {
    const int64_t row = static_cast<int64_t>(hd.b) * p.T + t;
    const T* in = static_cast<const T*>(p.qkvg) + row * p.ld;
    const int64_t pos = base + t - hd.kv0;
    const int64_t pp = min(max(pos, static_cast<int64_t>(0)), static_cast<int64_t>(max(p.npos - 1, 0)));
    const float *cs = p.cos_t + pp * half, *sn = p.sin_t + pp * half;
    for (int i = threadIdx.x; i < p.dim; i += kRecThreads) {
      float q, k;
      load_rotated<T, 1>(in + hd.h * p.dim, i, p.rot, cs, sn, &q);
      load_rotated<T, 1>(in + Hd + hd.h * p.dim, i, p.rot, cs, sn, &k);
      qs[i] = q;
      ks[i] = pos < 0 ? 0.f : k * p.kscale;
    }
    for (int i = threadIdx.x; i < p.vdim; i += kRecThreads) vs[i] = pos < 0 ? 0.f : to_f<T>(in[2 * Hd + hd.h * p.vdim + i]);
    __syncthreads();
    const bool zero = p.fresh && t == 0;
    for (int r0 = vlo + grp; r0 < vhi; r0 += ngrp * U) {
      float acc[U];
#pragma unroll
      for (int u = 0; u < U; ++u) acc[u] = 0.f;
      for (int i = li * VEC; i < p.dim; i += lpr * VEC) {
        float s[U][VEC];
#pragma unroll
        for (int u = 0; u < U; ++u) {
          const int v = r0 + u * ngrp;
#pragma unroll
          for (int e = 0; e < VEC; ++e) s[u][e] = 0.f;
          if (v < vhi && !zero) load_vec<float, VEC>(S + static_cast<int64_t>(v) * p.dim + i, s[u]);
        }
#pragma unroll
        for (int u = 0; u < U; ++u) {
          const int v = r0 + u * ngrp;
          if (v >= vhi) continue;
#pragma unroll
          for (int e = 0; e < VEC; ++e) {
            s[u][e] = dec * s[u][e] + ks[i + e] * vs[v];
            acc[u] += s[u][e] * qs[i + e];
          }
          store_vec<float, VEC>(S + static_cast<int64_t>(v) * p.dim + i, s[u]);
        }
      }
#pragma unroll
      for (int u = 0; u < U; ++u) {
        for (int o = lpr >> 1; o > 0; o >>= 1) acc[u] += __shfl_xor(acc[u], o, 64);
        const int v = r0 + u * ngrp;
        if (li == 0 && v < vhi) {
          if (p.vsplit > 1)
            __hip_atomic_store(&p.osplit[(static_cast<int64_t>(hd.b) * p.H + hd.h) * p.vdim + v], acc[u], __ATOMIC_RELAXED,
                               __HIP_MEMORY_SCOPE_AGENT);
          else
            os[v] = acc[u];
        }
      }
    }
    if (p.vsplit > 1) {  // (T == 1)
      __shared__ int last;
      asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
      __syncthreads();
      if (threadIdx.x == 0) {
        int* cnt = p.cnt + static_cast<int64_t>(hd.b) * p.H + hd.h;
        last = __hip_atomic_fetch_add(cnt, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == p.vsplit - 1;
        if (last) {
          __hip_atomic_store(cnt, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
          __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "agent");
          asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        }
      }
      __syncthreads();
      if (!last) return;
      for (int v = threadIdx.x; v < p.vdim; v += kRecThreads)
        os[v] = p.osplit[(static_cast<int64_t>(hd.b) * p.H + hd.h) * p.vdim + v];
    }
    __syncthreads();
    float ss = 0.f;
    for (int v = threadIdx.x; v < p.vdim; v += kRecThreads) ss += os[v] * os[v];
    const float rs = rsqrtf(block_sum<kRecThreads>(ss, scratch) / p.vdim + p.eps);
    for (int v = threadIdx.x; v < p.vdim; v += kRecThreads) {
      const float gv = to_f<T>(in[2 * Hd + Hv + hd.h * p.vdim + v]);
      static_cast<T*>(p.y)[row * Hv + hd.h * p.vdim + v] = from_f<T>(os[v] * rs * (gv / (1.f + expf(-gv))));
    }
    __syncthreads();
  }
}

constexpr int kLdsMax = 160 * 1024;

template <typename T>
int64_t state_lds(const RetentionParams& p, int C) {
  const int dp = round_up(p.dim, 32), vp = round_up(p.vdim, 16);
  return static_cast<int64_t>(sizeof(T)) * (Mma<T>::PL * dp + vp) * (C + pad16<T>());
}
template <typename T>
int64_t output_lds(const RetentionParams& p, int C) {
  const int dp = round_up(p.dim, 32), vp = round_up(p.vdim, 16), pd = pad16<T>();
  return static_cast<int64_t>(sizeof(T)) * (Mma<T>::PL * C * (dp + pd) + ret_k_elems(C, dp, Mma<T>::PL, pd) +
                                            vp * (C + pd)) + 4ll * C * (vp + 4);
}

template <typename T>
bool vec_ok(const RetentionParams& p) {
  return p.dim % 8 == 0 && p.vdim % 8 == 0 && p.rot % 16 == 0 && p.ld % 8 == 0 &&
         reinterpret_cast<uintptr_t>(p.qkvg) % 16 == 0;
}

template <typename K>
void allow_lds(K kernel, int64_t bytes) {
  if (bytes > 64 * 1024)
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize,
                              static_cast<int>(bytes));
}

void scan(const RetentionParams& p, hipStream_t st) {
  const int64_t n = static_cast<int64_t>(p.vdim) * p.dim;
  if (n % 4 == 0) ret_scan_kernel<4><<<dim3((n / 4 + 255) / 256, p.H, p.B), 256, 0, st>>>(p);
  else ret_scan_kernel<1><<<dim3((n + 255) / 256, p.H, p.B), 256, 0, st>>>(p);
}

template <typename T, int VEC>
void prefill(const RetentionParams& p, hipStream_t st) {
  const dim3 g(p.nc, p.H, p.B);
  const int64_t la = state_lds<T>(p, p.chunk), lc = output_lds<T>(p, p.chunk);
  allow_lds(ret_state_kernel<T, VEC>, la);
  ret_state_kernel<T, VEC><<<g, 256, la, st>>>(p);
  scan(p, st);
  if (p.chunk == 64) {
    allow_lds(ret_output_kernel<T, VEC, 4>, lc);
    ret_output_kernel<T, VEC, 4><<<g, 256, lc, st>>>(p);
  } else {
    allow_lds(ret_output_kernel<T, VEC, 2>, lc);
    ret_output_kernel<T, VEC, 2><<<g, 256, lc, st>>>(p);
  }
}

template <typename T>
void recurrent(const RetentionParams& p, hipStream_t st) {
  const bool v4 = p.dim % 4 == 0;
  int lpr = 1;
  while (lpr < 64 && lpr * (v4 ? 4 : 1) < p.dim) lpr *= 2;
  const int64_t lds = 4ll * (2 * round_up(p.dim, 4) + 2 * p.vdim);
  const dim3 g(p.H, p.B, p.vsplit);
  if (v4) ret_recurrent_kernel<T, 4><<<g, kRecThreads, lds, st>>>(p, lpr);
  else ret_recurrent_kernel<T, 1><<<g, kRecThreads, lds, st>>>(p, lpr);
}

template <typename T>
int pick_chunk(const RetentionParams& p) {
  for (int C = 64; C >= 32; C /= 2)
    if (output_lds<T>(p, C) <= kLdsMax && state_lds<T>(p, C) <= kLdsMax) return C;
  return 0;
}

}  // namespace

// chunk length of the chunked form, 0 if the recurrence takes the portion
int retention_chunk(bool bf16, const RetentionParams& p) {
  if (p.T < 16) return 0;
  if (bf16 && retention_mfma_ok(p)) return 128;
  return bf16 ? pick_chunk<bf16_t>(p) : pick_chunk<float>(p);
}

void launch_retention_prefill(bool bf16, const RetentionParams& p, hipStream_t st) {
  if (p.chunk == 128) {  // (bf16, retention_mfma_ok)
    launch_retention_state_mfma(p, st);
    scan(p, st);
    launch_retention_output_mfma(p, st);
  } else if (bf16) {
    if (vec_ok<bf16_t>(p)) prefill<bf16_t, 8>(p, st);
    else prefill<bf16_t, 1>(p, st);
  } else {
    if (vec_ok<float>(p)) prefill<float, 8>(p, st);
    else prefill<float, 1>(p, st);
  }
}

void launch_retention_recurrent(bool bf16, const RetentionParams& p, hipStream_t st) {
  if (bf16) recurrent<bf16_t>(p, st);
  else recurrent<float>(p, st);
}

}  // namespace dla
