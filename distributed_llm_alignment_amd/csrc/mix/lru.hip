// Real-gated linear recurrent unit behind a causal depthwise convolution, for gfx950.
//
//   u = conv(x + bias) (zeros before the start),  r, i = sigmoid(block-diagonal products of u)
//   log a = -c r softplus(lam),  S_t = a_t S_(t-1) + sqrt(1 - a_t^2) i_t u_t,  out = S * gelu_tanh(y + bias)
//
// Prompt portions, three launches:
//   gates   workgroup = (chunk of tokens, gate block or 128 channels of a large one, sequence): the
//           convolution of the block's channels goes to LDS, both gates' products run on MFMA with a
//           channel per lane column, and the chunk is scanned in registers (4 tokens per lane, two
//           shuffle steps per 16 tokens). Written: the state with the chunk started at zero, and the
//           product of decays.
//   scan    state at every chunk's start (one thread per sequence and channel); the convolution's ring
//   output  (local state + product of decays * start state) * gelu branch, elementwise
// Decode: one launch, workgroup = 16 channels x 16 rows, the block's input channels split over 4 waves.
//
// u is rounded to the compute dtype (it is an MFMA operand); gates, decays and states are fp32.
#include "mix_params.h"
#include "mma.h"

namespace dla {
namespace {

constexpr int kTT = 64;    // tokens per tile
constexpr int kNC = 128;   // channels a workgroup takes, or half of them
constexpr int kKC = 256;   // gate-block inputs staged at a time

template <typename T>
constexpr int pad16() { return 16 / static_cast<int>(sizeof(T)); }

__device__ __forceinline__ float sigm(float x) { return __builtin_amdgcn_rcpf(1.f + __expf(-x)); }
__device__ __forceinline__ float softplus(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
// 1 - e^x for x <= 0, without cancellation near zero
__device__ __forceinline__ float one_minus_exp(float x) {
  if (x < -0.5f) return 1.f - __expf(x);
  return -x * (1.f + x * (1.f / 2) * (1.f + x * (1.f / 3) * (1.f + x * (1.f / 4) * (1.f + x * (1.f / 5) * (1.f + x * (1.f / 6) * (1.f + x * (1.f / 7)))))));
}

// decay and input of one step; lam_c = -c softplus(lam)
__device__ __forceinline__ void lru_step(float zr, float zi, float u, float lam_c, float& a, float& b) {
  const float la = lam_c * sigm(zr);
  a = __expf(la);
  b = __builtin_amdgcn_sqrtf(one_minus_exp(2.f * la)) * sigm(zi) * u;
}

// convolution output of channel `ch` at column `col` (position pos >= 0), rounded to T; xrow(j): the raw
// projected x of column col - j
template <typename T, typename F>
__device__ __forceinline__ float conv_at(const LruParams& p, int ch, int64_t pos, F xrow) {
  const T* w = static_cast<const T*>(p.conv_w) + static_cast<int64_t>(ch) * p.taps;
  const float xb = to_f<T>(static_cast<const T*>(p.bias)[p.W + ch]);
  float s = to_f<T>(static_cast<const T*>(p.conv_b)[ch]);
  for (int j = 0; j < p.taps; ++j)
    if (pos >= j) s += to_f<T>(w[p.taps - 1 - j]) * (to_f<T>(xrow(j)) + xb);
  return to_f<T>(from_f<T>(s));
}

// The same for V channels ch .. ch + V - 1 (V divides ch) and consecutive columns, bf16, TAPS taps: `row(j)` is the
// raw x row of column col0 + j (j >= -(TAPS - 1)), pos0 the position of column col0; emits u of n columns.
template <int TAPS, int V, typename F, typename G>
__device__ __forceinline__ void conv_run(const LruParams& p, int ch, int64_t pos0, int n, F row, G emit) {
  float w[V][TAPS], xb[V], cb[V], win[TAPS][V];
  {
    const bf16_t* src = static_cast<const bf16_t*>(p.conv_w) + static_cast<int64_t>(ch) * TAPS;
    float v[TAPS][V];
#pragma unroll
    for (int i = 0; i < TAPS; ++i) load_vec<bf16_t, V>(src + V * i, v[i]);
#pragma unroll
    for (int e = 0; e < V; ++e)
#pragma unroll
      for (int j = 0; j < TAPS; ++j) w[e][j] = v[(e * TAPS + j) / V][(e * TAPS + j) % V];
    load_vec<bf16_t, V>(static_cast<const bf16_t*>(p.bias) + p.W + ch, xb);
    load_vec<bf16_t, V>(static_cast<const bf16_t*>(p.conv_b) + ch, cb);
  }
  auto fetch = [&](int j, float* o) {  // biased x of column col0 + j, zero before the start
    if (pos0 + j >= 0) {
      load_vec<bf16_t, V>(row(j), o);
#pragma unroll
      for (int e = 0; e < V; ++e) o[e] += xb[e];
    } else {
#pragma unroll
      for (int e = 0; e < V; ++e) o[e] = 0.f;
    }
  };
#pragma unroll
  for (int j = 0; j < TAPS - 1; ++j) fetch(j - (TAPS - 1), win[j + 1]);
#pragma unroll V == 4 ? 4 : 2
  for (int t = 0; t < n; ++t) {
#pragma unroll
    for (int j = 0; j < TAPS - 1; ++j)
#pragma unroll
      for (int e = 0; e < V; ++e) win[j][e] = win[j + 1][e];
    fetch(t, win[TAPS - 1]);
    float u[V];
#pragma unroll
    for (int e = 0; e < V; ++e) {
      u[e] = cb[e];
#pragma unroll
      for (int j = 0; j < TAPS; ++j) u[e] += w[e][j] * win[j][e];
      if (pos0 + t < 0) u[e] = 0.f;
    }
    emit(t, u);
  }
}

// 16 x KS gate-weight fragment: row `ch` of one gate block, inputs k ..
template <typename T, bool VEC>
__device__ __forceinline__ typename Mma<T>::Frag gate_frag(const T* wb, int n, int ch, int k) {
  using M = Mma<T>;
  auto f = M::zero();
  if (ch >= n) return f;
  const T* row = wb + static_cast<int64_t>(ch) * n + k;
  if constexpr (VEC) {
    if (k < n) f = M::row(row);
  } else {
#pragma unroll
    for (int e = 0; e < M::KV; ++e)
      if (k + e < n) M::set(f, e, row[e]);
  }
  return f;
}

// grid (nc, nb * ceil(n / (128 JG)), B), 256 threads, 128 JG channels (ONE: n <= kKC, a tile of tokens is
// staged once; JG > 1 only then). TAPS > 0: bf16, n % 8 == 0.
template <typename T, bool VEC, int TAPS, int JG, bool ONE>
__global__ __launch_bounds__(256, ONE ? 4 : 2) void lru_gates_kernel(LruParams p) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  using M = Mma<T>;
  constexpr int MT = kTT / 16, NJ = JG * kNC / 64, JA = ONE ? 1 : NJ;
  const int nblk = (p.n + kNC * JG - 1) / (kNC * JG);
  const int b = blockIdx.z, blk = blockIdx.y / nblk, c0 = (blockIdx.y % nblk) * kNC * JG;
  const int kc = min(kKC, round_up(p.n, 32)), ldu = kc + pad16<T>();
  T* us = reinterpret_cast<T*>(smem);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane & 15, g = lane >> 4;
  const int kv0 = p.kv_start ? p.kv_start[b] : 0;
  const T* X = static_cast<const T*>(p.yx) + static_cast<int64_t>(b) * p.T * 2 * p.W + p.W + blk * p.n;
  const T* Hs = static_cast<const T*>(p.hist) + static_cast<int64_t>(b) * p.taps * p.W + blk * p.n;
  const T* Wr = static_cast<const T*>(p.gates) + static_cast<int64_t>(blk) * p.n * p.n;
  const T* Wi = static_cast<const T*>(p.gates) + static_cast<int64_t>(p.nb + blk) * p.n * p.n;
  __shared__ float prm[3][kNC * JG], carry[2][kNC * JG];  // per channel: -c softplus(lam), gate biases; A, S so far
  for (int i = threadIdx.x; i < kNC * JG; i += 256) {
    const int ch = min(c0 + i, p.n - 1);
    prm[0][i] = -p.c * softplus(to_f<T>(static_cast<const T*>(p.lam)[blk * p.n + ch]));
    prm[1][i] = to_f<T>(static_cast<const T*>(p.gates_b)[blk * p.n + ch]);
    prm[2][i] = to_f<T>(static_cast<const T*>(p.gates_b)[(p.nb + blk) * p.n + ch]);
    carry[0][i] = 1.f;
    carry[1][i] = 0.f;
  }
  auto stage = [&](int t0, int k0) {
    if constexpr (TAPS > 0) {
      constexpr int V = 4;
      const int ng = kc / V, ntg = 256 / ng, per = (kTT + ntg - 1) / ntg;
      const int k = static_cast<int>(threadIdx.x) % ng * V, tg = threadIdx.x / ng * per;
      const int n = min(min(per, kTT - tg), p.T - t0 - tg);  // columns of this thread that exist
      const bool real = k0 + k < p.n;
      if (tg < kTT && real && n > 0) {
        const int64_t col = p.base + t0 + tg;
        conv_run<TAPS, V>(p, blk * p.n + k0 + k, col - kv0, n,
                          [&](int j) {
                            return t0 + tg + j >= 0 ? X + static_cast<int64_t>(t0 + tg + j) * 2 * p.W + k0 + k
                                                    : Hs + ((col + j) % TAPS) * p.W + k0 + k;
                          },
                          [&](int t, const float* u) { store_vec<bf16_t, V>(us + (tg + t) * ldu + k, u); });
      }
      const float z[V] = {0.f, 0.f, 0.f, 0.f};
      for (int t = real ? tg + max(n, 0) : tg; t < min(tg + per, kTT); ++t) store_vec<bf16_t, V>(us + t * ldu + k, z);
    } else {
      for (int i = threadIdx.x; i < kTT * kc; i += 256) {
        const int t = i / kc, k = i % kc;
        float v = 0.f;
        const int64_t col = p.base + t0 + t, pos = col - kv0;
        if (t0 + t < p.T && k0 + k < p.n && pos >= 0)
          v = conv_at<T>(p, blk * p.n + k0 + k, pos, [&](int j) {
            return t0 + t - j >= 0 ? X[static_cast<int64_t>(t0 + t - j) * 2 * p.W + k0 + k]
                                   : Hs[((col - j) % p.taps) * p.W + k0 + k];
          });
        us[t * ldu + k] = from_f<T>(v);
      }
    }
  };
  const int t_end = min((static_cast<int>(blockIdx.x) + 1) * p.chunk, p.T);
  for (int t0 = blockIdx.x * p.chunk; t0 < t_end; t0 += kTT) {
    if constexpr (ONE) {
      __syncthreads();  // every wave is done with the last tile
      stage(t0, 0);
      __syncthreads();
    }
    // the wave's 16-channel tiles; when a staged tile holds all inputs (ONE), one after the other
#pragma unroll 1
    for (int j0 = 0; j0 < NJ; j0 += JA) {
      f32x4 ar[JA][MT], ai[JA][MT];
      float u[JA][MT][4];
#pragma unroll
      for (int j = 0; j < JA; ++j)
#pragma unroll
        for (int m = 0; m < MT; ++m) {
          ar[j][m] = ai[j][m] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int i = 0; i < 4; ++i) u[j][m][i] = 0.f;
        }
      for (int k0 = 0; k0 < (ONE ? 1 : p.n); k0 += kc) {
        if constexpr (!ONE) {
          __syncthreads();
          stage(t0, k0);
          __syncthreads();
        }
#pragma unroll
        for (int j = 0; j < JA; ++j) {
          const int n0 = c0 + 16 * (wave + 4 * (j0 + j));
          if (n0 >= p.n) continue;
#pragma unroll 4
          for (int k = 0; k < kc; k += M::KS) {
            const auto fr = gate_frag<T, VEC>(Wr, p.n, n0 + r, k0 + k + g * M::KV);
            const auto fi = gate_frag<T, VEC>(Wi, p.n, n0 + r, k0 + k + g * M::KV);
#pragma unroll
            for (int m = 0; m < MT; ++m) {
              const auto a = M::row(us + (16 * m + r) * ldu + k + g * M::KV);
              ar[j][m] = M::mma(a, fr, ar[j][m]);
              ai[j][m] = M::mma(a, fi, ai[j][m]);
            }
          }
          const int kk = n0 + r - k0;  // this lane's own channel among the staged ones
          if (!ONE && kk >= 0 && kk < kc)
#pragma unroll
            for (int m = 0; m < MT; ++m)
#pragma unroll
              for (int i = 0; i < 4; ++i) u[j][m][i] = to_f<T>(us[(16 * m + 4 * g + i) * ldu + kk]);
        }
      }
#pragma unroll
      for (int j = 0; j < JA; ++j) {
        const int cl = 16 * (wave + 4 * (j0 + j)) + r, ch = c0 + cl;
        if (ch - r >= p.n) continue;
        const float lam_c = prm[0][cl], rb = prm[1][cl], ib = prm[2][cl];
        float ca = carry[0][cl], cs = carry[1][cl];
#pragma unroll
        for (int m = 0; m < MT; ++m) {
          // 4 tokens of this lane: A[i], S[i] = product of decays / state since the lane's first token
          float A[4], S[4], pa = 1.f, ps = 0.f;
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int t = t0 + 16 * m + 4 * g + i;
            float a, x;
            const float uv = ONE ? to_f<T>(us[(16 * m + 4 * g + i) * ldu + min(ch, kc - 1)]) : u[j][m][i];
            lru_step(ar[j][m][i] + rb, ai[j][m][i] + ib, uv, lam_c, a, x);
            const bool real = t < p.T && p.base + t >= kv0;
            a = real ? a : 1.f;
            ps = a * ps + (real ? x : 0.f);
            pa *= a;
            A[i] = pa;
            S[i] = ps;
          }
          // inclusive scan over the 4 lane groups, then what comes before this lane
#pragma unroll
          for (int o = 16; o <= 32; o <<= 1) {
            const float qa = __shfl_up(pa, o, 64), qs = __shfl_up(ps, o, 64);
            if (lane >= o) {
              ps = pa * qs + ps;
              pa *= qa;
            }
          }
          float ea = __shfl_up(pa, 16, 64), es = __shfl_up(ps, 16, 64);
          if (g == 0) {
            ea = 1.f;
            es = 0.f;
          }
          es = ea * cs + es;
          ea *= ca;
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int t = t0 + 16 * m + 4 * g + i;
            if (t < p.T && ch < p.n) {
              const int64_t at = (static_cast<int64_t>(b) * p.T + t) * p.W + blk * p.n + ch;
              p.cum[at] = ea * A[i];
              p.loc[at] = A[i] * es + S[i];
            }
          }
          const float la = __shfl(pa, 48 + r, 64), ls = __shfl(ps, 48 + r, 64);
          cs = la * cs + ls;
          ca *= la;
        }
        if (g == 0) {  // (channels of this wave alone: its LDS accesses stay in order)
          carry[0][cl] = ca;
          carry[1][cl] = cs;
        }
      }
    }
  }
}

// grid (ceil(W / 64), B), 64 threads: start[c] <- state at chunk c's start, state <- final state; the
// last `taps` x rows go into the ring
template <typename T>
__global__ __launch_bounds__(64) void lru_scan_kernel(LruParams p) {
  const int ch = blockIdx.x * 64 + threadIdx.x, b = blockIdx.y;
  if (ch >= p.W) return;
  const int64_t at = static_cast<int64_t>(b) * p.W + ch;
  float S = p.base > 0 ? p.state[at] : 0.f;
  constexpr int U = 16;
  for (int c0 = 0; c0 < p.nc; c0 += U) {
    float a[U], s[U];
#pragma unroll
    for (int i = 0; i < U; ++i) {
      if (c0 + i >= p.nc) break;
      const int64_t row = static_cast<int64_t>(b) * p.T + min((c0 + i + 1) * p.chunk, p.T) - 1;
      a[i] = p.cum[row * p.W + ch];
      s[i] = p.loc[row * p.W + ch];
    }
#pragma unroll
    for (int i = 0; i < U; ++i) {
      if (c0 + i >= p.nc) break;
      p.start[(static_cast<int64_t>(b) * p.nc + c0 + i) * p.W + ch] = S;
      S = a[i] * S + s[i];
    }
  }
  p.state[at] = S;
  const T* X = static_cast<const T*>(p.yx) + static_cast<int64_t>(b) * p.T * 2 * p.W + p.W + ch;
  T* Hs = static_cast<T*>(p.hist) + static_cast<int64_t>(b) * p.taps * p.W + ch;
  for (int t = max(0, p.T - p.taps); t < p.T; ++t) Hs[((p.base + t) % p.taps) * p.W] = X[static_cast<int64_t>(t) * 2 * p.W];
}

// grid (rows of VEC channels / 256, tokens / RT, B)
constexpr int kRT = 4;
template <typename T, int VEC>
__global__ __launch_bounds__(256) void lru_output_kernel(LruParams p) {
  const int ch = (blockIdx.x * 256 + threadIdx.x) * VEC, b = blockIdx.z;
  if (ch >= p.W) return;
  float yb[VEC];
  load_vec<T, VEC>(static_cast<const T*>(p.bias) + ch, yb);
  const int t0 = blockIdx.y * kRT;
  float S[kRT][VEC], a[kRT][VEC], s[kRT][VEC], y[kRT][VEC];
#pragma unroll
  for (int i = 0; i < kRT; ++i) {
    const int t = min(t0 + i, p.T - 1);
    const int64_t row = static_cast<int64_t>(b) * p.T + t;
    load_vec<float, VEC>(p.start + (static_cast<int64_t>(b) * p.nc + t / p.chunk) * p.W + ch, S[i]);
    load_vec<float, VEC>(p.cum + row * p.W + ch, a[i]);
    load_vec<float, VEC>(p.loc + row * p.W + ch, s[i]);
    load_vec<T, VEC>(static_cast<const T*>(p.yx) + row * 2 * p.W + ch, y[i]);
  }
#pragma unroll
  for (int i = 0; i < kRT; ++i) {
    if (t0 + i >= p.T) break;
#pragma unroll
    for (int e = 0; e < VEC; ++e) s[i][e] = (s[i][e] + a[i][e] * S[i][e]) * gelu_tanh(y[i][e] + yb[e]);
    store_vec<T, VEC>(static_cast<T*>(p.out) + (static_cast<int64_t>(b) * p.T + t0 + i) * p.W + ch, s[i]);
  }
}

// grid (nb * ceil(n / 16), ceil(B / 16)), 256 threads. TAPS > 0: bf16, n % 8 == 0.
constexpr int kDK = 1024;  // gate-block inputs staged at a time
template <typename T, bool VEC, int TAPS>
__global__ __launch_bounds__(256) void lru_decode_kernel(LruParams p) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  __shared__ float red[2][4][4][64];
  using M = Mma<T>;
  const int nt = (p.n + 15) / 16, blk = blockIdx.x / nt, n0 = (blockIdx.x % nt) * 16, b0 = blockIdx.y * 16;
  const int kc = min(kDK, round_up(p.n, 32)), ldu = kc + pad16<T>();
  T* us = reinterpret_cast<T*>(smem);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane & 15, g = lane >> 4;
  const int nr = min(16, p.B - b0);
  const T* Wr = static_cast<const T*>(p.gates) + static_cast<int64_t>(blk) * p.n * p.n;
  const T* Wi = static_cast<const T*>(p.gates) + static_cast<int64_t>(p.nb + blk) * p.n * p.n;
  const T* YX = static_cast<const T*>(p.yx);
  T* Hs = static_cast<T*>(p.hist);
  const int ti = 4 * g + wave, ch = n0 + r;  // this thread's output: row ti, channel ch
  // the first weights leave before the convolution; the rest of the thread's operands with them
  constexpr int UK = 2;
  typename M::Frag fr[UK], fi[UK];
#pragma unroll
  for (int q = 0; q < UK; ++q) {
    const int k = (wave + 4 * q) * M::KS + g * M::KV;
    fr[q] = gate_frag<T, VEC>(Wr, p.n, ch, k);
    fi[q] = gate_frag<T, VEC>(Wi, p.n, ch, k);
  }
  const bool out = ti < nr && ch < p.n;
  const int c = blk * p.n + min(ch, p.n - 1), bo = b0 + min(ti, nr - 1);
  const int64_t at = static_cast<int64_t>(bo) * p.W + c;
  const float br = to_f<T>(static_cast<const T*>(p.gates_b)[c]), bi = to_f<T>(static_cast<const T*>(p.gates_b)[p.W + c]);
  const float lam = to_f<T>(static_cast<const T*>(p.lam)[c]), S0 = p.state[at];
  const T y0 = YX[static_cast<int64_t>(bo) * 2 * p.W + c], x0 = YX[static_cast<int64_t>(bo) * 2 * p.W + p.W + c];
  const float yb = to_f<T>(static_cast<const T*>(p.bias)[c]);
  const int64_t col = p.slot[0];
  f32x4 ar = {0.f, 0.f, 0.f, 0.f}, ai = ar;
  float uo = 0.f;
  for (int k0 = 0; k0 < p.n; k0 += kc) {
    if (k0) __syncthreads();
    if constexpr (TAPS > 0) {
      for (int i = threadIdx.x; i < 16 * (kc / 8); i += 256) {
        const int m = i / (kc / 8), k = i % (kc / 8) * 8, b = b0 + m;
        if (m < nr && k0 + k < p.n) {
          const int cc = blk * p.n + k0 + k;
          conv_run<TAPS, 8>(p, cc, col - (p.kv_start ? p.kv_start[b] : 0), 1,
                            [&](int j) {
                              return j == 0 ? YX + static_cast<int64_t>(b) * 2 * p.W + p.W + cc
                                            : Hs + (static_cast<int64_t>(b) * TAPS + (col + j) % TAPS) * p.W + cc;
                            },
                            [&](int, const float* u) { store_vec<bf16_t, 8>(us + m * ldu + k, u); });
        } else {
          store_bf16x8(us + m * ldu + k, bf16x8{0, 0, 0, 0, 0, 0, 0, 0});
        }
      }
    } else {
      for (int i = threadIdx.x; i < 16 * kc; i += 256) {
        const int m = i / kc, k = i % kc;
        float v = 0.f;
        if (m < nr && k0 + k < p.n) {
          const int cc = blk * p.n + k0 + k, b = b0 + m;
          v = conv_at<T>(p, cc, col - (p.kv_start ? p.kv_start[b] : 0), [&](int j) {
            return j == 0 ? YX[static_cast<int64_t>(b) * 2 * p.W + p.W + cc]
                          : Hs[(static_cast<int64_t>(b) * p.taps + (col - j) % p.taps) * p.W + cc];
          });
        }
        us[m * ldu + k] = from_f<T>(v);
      }
    }
    __syncthreads();
    int q = 0;
#pragma unroll
    for (int k = wave * M::KS; k < kc; k += 4 * M::KS, ++q) {
      const auto a = M::row(us + r * ldu + k + g * M::KV);
      const bool have = k0 == 0 && q < UK;
      auto wr = q == 0 ? fr[0] : fr[1], wi = q == 0 ? fi[0] : fi[1];
      if (!have) {
        wr = gate_frag<T, VEC>(Wr, p.n, ch, k0 + k + g * M::KV);
        wi = gate_frag<T, VEC>(Wi, p.n, ch, k0 + k + g * M::KV);
      }
      ar = M::mma(a, wr, ar);
      ai = M::mma(a, wi, ai);
    }
    if (ch - k0 >= 0 && ch - k0 < kc) uo = to_f<T>(us[ti * ldu + ch - k0]);
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    red[0][wave][i][lane] = ar[i];
    red[1][wave][i][lane] = ai[i];
  }
  __syncthreads();
  if (!out) return;  // (register i = wave of every wave's tile: row 4 g + wave)
  float zr = br, zi = bi;
#pragma unroll
  for (int w = 0; w < 4; ++w) {
    zr += red[0][w][wave][lane];
    zi += red[1][w][wave][lane];
  }
  float a, x;
  lru_step(zr, zi, uo, -p.c * softplus(lam), a, x);
  const float S = a * S0 + x;
  p.state[at] = S;
  Hs[(static_cast<int64_t>(bo) * p.taps + col % p.taps) * p.W + c] = x0;
  static_cast<T*>(p.out)[at] = from_f<T>(S * gelu_tanh(to_f<T>(y0) + yb));
}

// multiples of 128 channels per workgroup
int lru_passes(const LruParams& p) { return p.n > kNC && p.n <= kKC ? 2 : 1; }

template <typename K>
void allow_lds(K kernel, int64_t bytes) {
  if (bytes > 64 * 1024)
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize,
                              static_cast<int>(bytes));
}

bool gates_vec(const LruParams& p) { return p.n % 8 == 0 && reinterpret_cast<uintptr_t>(p.gates) % 16 == 0; }

// taps of the vectorised convolution, 0: element by element
int conv_taps(bool bf16, const LruParams& p) {
  const auto al = [](const void* x) { return reinterpret_cast<uintptr_t>(x) % 16 == 0; };
  const bool ok = bf16 && gates_vec(p) && p.taps >= 2 && p.taps <= 4 && al(p.yx) && al(p.bias) && al(p.conv_w) && al(p.conv_b) &&
                  al(p.hist);
  return ok ? p.taps : 0;
}

template <typename T, bool VEC, int TAPS, int JG, bool ONE>
void gates(const LruParams& p, hipStream_t st) {
  const dim3 g(p.nc, p.nb * ((p.n + kNC * JG - 1) / (kNC * JG)), p.B);
  const int kc = p.n < kKC ? round_up(p.n, 32) : kKC;
  const int64_t lds = static_cast<int64_t>(sizeof(T)) * kTT * (kc + pad16<T>());
  allow_lds(lru_gates_kernel<T, VEC, TAPS, JG, ONE>, lds);
  lru_gates_kernel<T, VEC, TAPS, JG, ONE><<<g, 256, lds, st>>>(p);
}
template <typename T, bool VEC, int TAPS>
void gates(const LruParams& p, hipStream_t st) {
  if (lru_passes(p) == 2) gates<T, VEC, TAPS, 2, true>(p, st);
  else if (p.n <= kKC) gates<T, VEC, TAPS, 1, true>(p, st);
  else gates<T, VEC, TAPS, 1, false>(p, st);
}

template <typename T>
void prefill(const LruParams& p, hipStream_t st) {
  if constexpr (sizeof(T) == 2) {
    const int taps = conv_taps(true, p);
    if (taps == 4) gates<T, true, 4>(p, st);
    else if (taps == 3) gates<T, true, 3>(p, st);
    else if (taps == 2) gates<T, true, 2>(p, st);
    else if (gates_vec(p)) gates<T, true, 0>(p, st);
    else gates<T, false, 0>(p, st);
  } else {
    if (gates_vec(p)) gates<T, true, 0>(p, st);
    else gates<T, false, 0>(p, st);
  }
  lru_scan_kernel<T><<<dim3((p.W + 63) / 64, p.B), 64, 0, st>>>(p);
  const auto al = [](const void* x) { return reinterpret_cast<uintptr_t>(x) % 16 == 0; };
  const unsigned ty = (p.T + kRT - 1) / kRT;
  if (p.W % 4 == 0 && al(p.yx) && al(p.out) && al(p.bias) && al(p.cum) && al(p.loc) && al(p.start))
    lru_output_kernel<T, 4><<<dim3((p.W / 4 + 255) / 256, ty, p.B), 256, 0, st>>>(p);
  else
    lru_output_kernel<T, 1><<<dim3((p.W + 255) / 256, ty, p.B), 256, 0, st>>>(p);
}

template <typename T, bool VEC, int TAPS>
void step(const LruParams& p, hipStream_t st) {
  const dim3 g(p.nb * ((p.n + 15) / 16), (p.B + 15) / 16);
  const int kc = p.n < kDK ? round_up(p.n, 32) : kDK;
  const int64_t lds = static_cast<int64_t>(sizeof(T)) * 16 * (kc + pad16<T>());
  allow_lds(lru_decode_kernel<T, VEC, TAPS>, lds);
  lru_decode_kernel<T, VEC, TAPS><<<g, 256, lds, st>>>(p);
}

template <typename T>
void decode(const LruParams& p, hipStream_t st) {
  if constexpr (sizeof(T) == 2) {
    const int taps = conv_taps(true, p);
    if (taps == 4) step<T, true, 4>(p, st);
    else if (taps == 3) step<T, true, 3>(p, st);
    else if (taps == 2) step<T, true, 2>(p, st);
    else if (gates_vec(p)) step<T, true, 0>(p, st);
    else step<T, false, 0>(p, st);
  } else {
    if (gates_vec(p)) step<T, true, 0>(p, st);
    else step<T, false, 0>(p, st);
  }
}

}  // namespace

// tokens per chunk: enough workgroups for the chip, few chunks to scan
int lru_chunk(const LruParams& p) {
  const int nc = kNC * lru_passes(p);
  const int64_t per = static_cast<int64_t>(p.nb) * ((p.n + nc - 1) / nc) * p.B;
  int c = 4 * kTT;
  while (c > kTT && per * ((p.T + c - 1) / c) < 1024) c /= 2;
  return c;
}

void launch_lru_prefill(bool bf16, const LruParams& p, hipStream_t st) {
  if (bf16) prefill<bf16_t>(p, st);
  else prefill<float>(p, st);
}

void launch_lru_decode(bool bf16, const LruParams& p, hipStream_t st) {
  if (bf16) decode<bf16_t>(p, st);
  else decode<float>(p, st);
}

}  // namespace dla
