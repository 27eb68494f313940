// Decode projections on the fp32 residual stream (few rows): y = epilogue(rowscale o (a W^T)), bf16 a [M, K],
// W [N, K], M <= 32. One workgroup = 16 output columns, 8 waves over K (in-workgroup split, summed
// in wave order), as csrc/skinny_ks.h; what is different is the epilogue side:
//
//   kStore    y = bf16
//   kRelu2    y = bf16(relu(.)^2)
//   kGate     y = bf16(gelu_tanh(.) * table[ids[m], off + n])
//   kStream   x[m, n] += .   (fp32 stream, in place);  y = bf16(x * (offset + norm_w[n])), or bf16(x);
//             ssq[m, block] = sum of x^2 over the block's 16 columns
//
// A norm between two projections costs no launch: the producer (kStream) writes x * (offset + w)
// and the partial sums of squares, the consumer scales its rows by rsqrt(mean(x^2) + eps) (`ssq_in`).
#include "mix_params.h"
#include "mma.h"

namespace dla {
namespace {

enum { kStore = 0, kRelu2 = 1, kGate = 2, kStream = 3 };
constexpr int kWaves = 8, kU = 4;

template <int MT, int EPI>
__global__ __launch_bounds__(64 * kWaves) void stream_gemm_kernel(StreamGemmParams p) {
  __shared__ float red[kWaves][4 * MT][64];
  __shared__ float rstd[16 * MT];
  using M = Mma<bf16_t>;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane & 15, g = lane >> 4;
  const int n0 = blockIdx.x * 16;
  const int steps = (p.K + 31) / 32, per = (steps + kWaves - 1) / kWaves;
  const int s0 = wave * per, s1 = min(s0 + per, steps);
  const bf16_t* W = p.w + static_cast<int64_t>(min(n0 + r, p.N - 1)) * p.K;
  const bf16_t* A[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) A[t] = p.a + static_cast<int64_t>(min(16 * t + r, p.M - 1)) * p.K;
  s16x8 wf[2][kU], af[2][kU][MT];
  auto load = [&](int buf, int s) {
#pragma unroll
    for (int u = 0; u < kU; ++u) {
      const int k = 32 * (s + u) + 8 * g;
      const bool in = s + u < s1 && k < p.K;
      const int kc = in ? k : 0;
      wf[buf][u] = M::row(W + kc);
#pragma unroll
      for (int t = 0; t < MT; ++t) {
        const s16x8 v = M::row(A[t] + kc);
        af[buf][u][t] = in ? v : M::zero();
      }
    }
  };
  f32x4 acc[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  if (s0 < s1) load(0, s0);
  if (p.ssq_in) {
    for (int m = wave; m < p.M; m += kWaves) {
      float v = 0.f;
      for (int i = lane; i < p.nssq; i += 64) v += p.ssq_in[static_cast<int64_t>(m) * p.nssq + i];
      v = wave_sum(v);
      if (lane == 0) rstd[m] = rsqrtf(v / p.K + p.eps);
    }
  }
  for (int s = s0; s < s1; s += 2 * kU) {
    if (s + kU < s1) load(1, s + kU);
#pragma unroll
    for (int u = 0; u < kU; ++u)
#pragma unroll
      for (int t = 0; t < MT; ++t) acc[t] = M::mma(af[0][u][t], wf[0][u], acc[t]);
    if (s + kU < s1) {
      if (s + 2 * kU < s1) load(0, s + 2 * kU);
#pragma unroll
      for (int u = 0; u < kU; ++u)
#pragma unroll
        for (int t = 0; t < MT; ++t) acc[t] = M::mma(af[1][u][t], wf[1][u], acc[t]);
    }
  }
#pragma unroll
  for (int t = 0; t < MT; ++t)
#pragma unroll
    for (int i = 0; i < 4; ++i) red[wave][4 * t + i][lane] = acc[t][i];
  __syncthreads();
  const int ti = threadIdx.x >> 6;  // 4 t + i, one per wave
  if (ti >= 4 * MT) return;
  const int m = 16 * (ti >> 2) + 4 * g + (ti & 3), n = n0 + r;
  float v = 0.f;
#pragma unroll
  for (int w = 0; w < kWaves; ++w) v += red[w][ti][lane];
  const bool ok = m < p.M && n < p.N;
  if (p.ssq_in) v *= rstd[min(m, p.M - 1)];
  const int64_t at = static_cast<int64_t>(m) * p.N + n;
  if constexpr (EPI == kRelu2) {
    v = fmaxf(v, 0.f);
    v *= v;
  }
  if constexpr (EPI == kGate) {
    if (ok) {
      const int64_t id = p.ids[m];
      const float e = id >= 0 && id < p.vocab ? bf2f(p.table[id * p.ldt + p.off + n]) : 0.f;
      v = gelu_tanh(v) * e;
    }
  }
  if constexpr (EPI == kStream) {
    float sq = 0.f;
    if (ok) {
      const float x = p.x[at] + v;
      p.x[at] = x;
      sq = x * x;
      v = p.norm_w ? x * (p.offset + bf2f(p.norm_w[n])) : x;
    }
#pragma unroll
    for (int o = 1; o < 16; o <<= 1) sq += __shfl_xor(sq, o, 64);
    if (r == 0 && m < p.M) p.ssq[static_cast<int64_t>(m) * gridDim.x + blockIdx.x] = sq;
  }
  if (ok) p.y[at] = f2bf(v);
}

template <int MT>
void go(const StreamGemmParams& p, int epi, hipStream_t st) {
  const dim3 g((p.N + 15) / 16);
  if (epi == kStore) stream_gemm_kernel<MT, kStore><<<g, 64 * kWaves, 0, st>>>(p);
  else if (epi == kRelu2) stream_gemm_kernel<MT, kRelu2><<<g, 64 * kWaves, 0, st>>>(p);
  else if (epi == kGate) stream_gemm_kernel<MT, kGate><<<g, 64 * kWaves, 0, st>>>(p);
  else stream_gemm_kernel<MT, kStream><<<g, 64 * kWaves, 0, st>>>(p);
}

}  // namespace

void launch_stream_gemm(const StreamGemmParams& p, int epi, hipStream_t st) {
  if (p.M <= 16) go<1>(p, epi, st);
  else go<2>(p, epi, st);
}

}  // namespace dla
