// Gated linear attention (linear attention with a decay per key channel and token) for gfx950.
//
//   log alpha = log sigmoid(a2 (a1 h) + b) / tau
//   S_t = diag(alpha_t) S_(t-1) + k_t v_t^T,  o_t = S_t^T q_t dim^(-1/2),  y = o / rms(o) * w * silu(g)
//
// This file: the recurrence itself, token by token, for decode, short portions, fp32 and head sizes
// that the chunked form (gla_mfma.hip) does not take. One workgroup per (sequence, head) reads and
// writes its state once per token; decode of few rows splits the value rows over workgroups, and the
// last to arrive does the norm and the gate (nobody waits for anybody).
//
// The state is kept transposed, [vdim, dim]: a row is what one output column needs, contiguous. The
// second decay product, decays, state and norm are fp32.
#include "mix_params.h"
#include "mma.h"

namespace dla {
namespace {

constexpr int kThreads = 512;

// log2 of a channel's decay
__device__ __forceinline__ float log2_decay(float z, float inv_tau) {
  constexpr float kLog2e = 1.4426950408889634f;
  return (fminf(z, 0.f) - log1pf(expf(-fabsf(z)))) * (inv_tau * kLog2e);
}

// grid (H, B, vsplit); a row of the state (one v) belongs to a group of `lpr` lanes, each lane to
// VEC-element pieces of it
template <typename T, int VEC>
__global__ __launch_bounds__(kThreads, 4) void gla_recurrent_kernel(GlaParams p, int lpr) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  __shared__ float scratch[kThreads / 64];
  const int d4 = round_up(p.dim, 4);
  float* qs = reinterpret_cast<float*>(smem);
  float* ks = qs + d4;
  float* as = ks + d4;  // decays
  float* vs = as + d4;
  float* os = vs + p.vdim;
  const int h = blockIdx.x, b = blockIdx.y;
  const int kv0 = p.kv_start ? p.kv_start[b] : 0;
  const int Hd = p.H * p.dim, Hv = p.H * p.vdim;
  const T* A2 = static_cast<const T*>(p.a2) + static_cast<int64_t>(h) * p.dim * p.rank;
  const T* A2b = static_cast<const T*>(p.a2_b) + h * p.dim;
  float* S = p.state + (static_cast<int64_t>(b) * p.H + h) * p.vdim * p.dim;
  const int grp = threadIdx.x / lpr, li = threadIdx.x % lpr, ngrp = kThreads / lpr;
  constexpr int U = 4;
  const int per = (p.vdim + p.vsplit - 1) / p.vsplit, vlo = blockIdx.z * per, vhi = min(vlo + per, p.vdim);
  auto load_state = [&](int r0, int i, float (&s)[U][VEC]) {  // VEC state elements of U value rows
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int v = r0 + u * ngrp;
#pragma unroll
      for (int e = 0; e < VEC; ++e) s[u][e] = 0.f;
      if (v < vhi && i < p.dim) load_vec<float, VEC>(S + static_cast<int64_t>(v) * p.dim + i, s[u]);
    }
  };
  const bool rank8 = p.rank % 8 == 0 && p.ld % 8 == 0 && (reinterpret_cast<uintptr_t>(p.proj) | reinterpret_cast<uintptr_t>(p.a2)) % 16 == 0 &&
                     (2 * (Hd + Hv)) % 8 == 0;
  for (int t = 0; t < p.T; ++t) {
    float pre[U][VEC];  // the first piece of the state is on its way while the decays are formed
    load_state(vlo + grp, li * VEC, pre);
    const int64_t row = static_cast<int64_t>(b) * p.T + t;
    const T* in = static_cast<const T*>(p.proj) + row * p.ld;
    const bool pad = p.base + t < kv0;
    for (int i = threadIdx.x; i < p.dim; i += kThreads) {
      float z = to_f<T>(A2b[i]);
      const T *w = A2 + static_cast<int64_t>(i) * p.rank, *a = in + 2 * (Hd + Hv);
      if (rank8) {
        for (int j = 0; j < p.rank; j += 8) {
          float x[8], y[8];
          load_vec<T, 8>(w + j, x);
          load_vec<T, 8>(a + j, y);
#pragma unroll
          for (int e = 0; e < 8; ++e) z += x[e] * y[e];
        }
      } else {
        for (int j = 0; j < p.rank; ++j) z += to_f<T>(w[j]) * to_f<T>(a[j]);
      }
      qs[i] = to_f<T>(in[h * p.dim + i]) * p.qscale;
      ks[i] = pad ? 0.f : to_f<T>(in[Hd + h * p.dim + i]);
      as[i] = pad ? 1.f : exp2f(log2_decay(z, p.inv_tau));
    }
    for (int i = threadIdx.x; i < p.vdim; i += kThreads) vs[i] = pad ? 0.f : to_f<T>(in[2 * Hd + h * p.vdim + i]);
    __syncthreads();
    const bool zero = p.fresh && t == 0;
    for (int r0 = vlo + grp; r0 < vhi; r0 += ngrp * U) {
      float acc[U];
#pragma unroll
      for (int u = 0; u < U; ++u) acc[u] = 0.f;
      for (int i = li * VEC; i < p.dim; i += lpr * VEC) {
        float s[U][VEC];
        if (r0 == vlo + grp && i == li * VEC) {
#pragma unroll
          for (int u = 0; u < U; ++u)
#pragma unroll
            for (int e = 0; e < VEC; ++e) s[u][e] = pre[u][e];
        } else {
          load_state(r0, i, s);
        }
#pragma unroll
        for (int u = 0; u < U; ++u) {
          const int v = r0 + u * ngrp;
          if (v >= vhi) continue;
#pragma unroll
          for (int e = 0; e < VEC; ++e) {
            if (zero) s[u][e] = 0.f;
            s[u][e] = as[i + e] * s[u][e] + ks[i + e] * vs[v];
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
            __hip_atomic_store(&p.osplit[(static_cast<int64_t>(b) * p.H + h) * p.vdim + v], acc[u], __ATOMIC_RELAXED,
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
        int* cnt = p.cnt + static_cast<int64_t>(b) * p.H + h;
        last = __hip_atomic_fetch_add(cnt, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == p.vsplit - 1;
        if (last) {
          __hip_atomic_store(cnt, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
          __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "agent");
          asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        }
      }
      __syncthreads();
      if (!last) return;
      for (int v = threadIdx.x; v < p.vdim; v += kThreads)
        os[v] = p.osplit[(static_cast<int64_t>(b) * p.H + h) * p.vdim + v];
    }
    __syncthreads();
    float ss = 0.f;
    for (int v = threadIdx.x; v < p.vdim; v += kThreads) ss += os[v] * os[v];
    const float rs = rsqrtf(block_sum<kThreads>(ss, scratch) / p.vdim + p.eps);
    for (int v = threadIdx.x; v < p.vdim; v += kThreads) {
      const float gv = to_f<T>(in[2 * Hd + Hv + h * p.vdim + v]), w = to_f<T>(static_cast<const T*>(p.norm_w)[v]);
      static_cast<T*>(p.y)[row * Hv + h * p.vdim + v] = from_f<T>(os[v] * rs * w * (gv / (1.f + expf(-gv))));
    }
    __syncthreads();
  }
}

template <typename T>
void recurrent(const GlaParams& p, hipStream_t st) {
  const bool v4 = p.dim % 4 == 0;
  int lpr = 1;
  while (lpr < 64 && lpr * (v4 ? 4 : 1) < p.dim) lpr *= 2;
  const int64_t lds = gla_recurrent_lds(p);
  const dim3 g(p.H, p.B, p.vsplit);
  if (v4) gla_recurrent_kernel<T, 4><<<g, kThreads, lds, st>>>(p, lpr);
  else gla_recurrent_kernel<T, 1><<<g, kThreads, lds, st>>>(p, lpr);
}

}  // namespace

void launch_gla_recurrent(bool bf16, const GlaParams& p, hipStream_t st) {
  if (bf16) recurrent<bf16_t>(p, st);
  else recurrent<float>(p, st);
}

}  // namespace dla
