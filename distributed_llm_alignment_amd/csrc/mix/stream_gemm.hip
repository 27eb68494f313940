// Decode projections on the fp32 residual stream (few rows): y = epilogue(rowscale o (a W^T)), bf16 a [M, K],
// W [N, K], M <= 32. One workgroup = 16 output columns, 8 waves over K (in-workgroup split, summed
// in wave order), as csrc/skinny_ks.h; what is different is the epilogue side:
//
//   kStore    y = bf16
//   kRelu2    y = bf16(relu(.)^2)
//   kGate     y = bf16(gelu_tanh(.) * table[ids[m], off + n])
//   kStream   x[m, n] += .   (fp32 stream, in place);  y = bf16(x * (offset + norm_w[n])), or bf16(x);
//             ssq[m, block] = sum of x^2 over the block's 16 columns
//   kPost     norms after the sums: x[m, n] holds the last sum, its norm x_prev = x * res_w * rstd(res_ssq) is
//             applied here; x <- alpha x_prev + . + bias;  y = bf16(x * norm_w[n]);  ssq as above
//   kGeglu    y = bf16(gelu_tanh(. gate) * . up), W = [gate rows; up rows]
//   kCap      y = fp32 cap * tanh(. / cap)
//
// A norm between two projections costs no launch: the producer (kStream, kPost) writes x * (offset + w)
// and the partial sums of squares, the consumer scales its rows by rsqrt(mean(x^2) + eps) (`ssq_in`).
#include "mix_params.h"
#include "mma.h"

namespace dla {
namespace {

enum { kStore = 0, kRelu2 = 1, kGate = 2, kStream = 3, kPost = 4, kGeglu = 5, kCap = 6 };
constexpr int kWaves = 8, kU = 4;

// 1 / rms of every row from partial sums of squares of K columns
__device__ __forceinline__ void row_scales(const float* ssq, int n, int M, int K, float eps, float* rstd) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  for (int m = wave; m < M; m += kWaves) {
    float v = 0.f;
    for (int i = lane; i < n; i += 64) v += ssq[static_cast<int64_t>(m) * n + i];
    v = wave_sum(v);
    if (lane == 0) rstd[m] = rsqrtf(v / K + eps);
  }
}

template <int MT, int EPI>
__global__ __launch_bounds__(64 * kWaves) void stream_gemm_kernel(StreamGemmParams p) {
  constexpr int NW = EPI == kGeglu ? 2 : 1;  // weight rows per output column
  __shared__ float red[kWaves][4 * MT * NW][64];
  __shared__ float rstd[16 * MT], rres[16 * MT];
  using M = Mma<bf16_t>;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane & 15, g = lane >> 4;
  const int n0 = blockIdx.x * 16;
  const int steps = (p.K + 31) / 32, per = (steps + kWaves - 1) / kWaves;
  const int s0 = wave * per, s1 = min(s0 + per, steps);
  const bf16_t* W[NW];
#pragma unroll
  for (int q = 0; q < NW; ++q) W[q] = p.w + static_cast<int64_t>(min(n0 + r, p.N - 1) + q * p.N) * p.K;
  const bf16_t* A[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) A[t] = p.a + static_cast<int64_t>(min(16 * t + r, p.M - 1)) * p.K;
  s16x8 wf[2][kU][NW], af[2][kU][MT];
  auto load = [&](int buf, int s) {
#pragma unroll
    for (int u = 0; u < kU; ++u) {
      const int k = 32 * (s + u) + 8 * g;
      const bool in = s + u < s1 && k < p.K;
      const int kc = in ? k : 0;
#pragma unroll
      for (int q = 0; q < NW; ++q) wf[buf][u][q] = M::row(W[q] + kc);
#pragma unroll
      for (int t = 0; t < MT; ++t) {
        const s16x8 v = M::row(A[t] + kc);
        af[buf][u][t] = in ? v : M::zero();
      }
    }
  };
  f32x4 acc[NW][MT];
#pragma unroll
  for (int q = 0; q < NW; ++q)
#pragma unroll
    for (int t = 0; t < MT; ++t) acc[q][t] = f32x4{0.f, 0.f, 0.f, 0.f};
  if (s0 < s1) load(0, s0);
  if (p.ssq_in) row_scales(p.ssq_in, p.nssq, p.M, p.K, p.eps, rstd);
  if constexpr (EPI == kPost) {
    if (p.res_ssq) row_scales(p.res_ssq, p.nres, p.M, p.N, p.eps, rres);
  }
  for (int s = s0; s < s1; s += 2 * kU) {
    if (s + kU < s1) load(1, s + kU);
#pragma unroll
    for (int u = 0; u < kU; ++u)
#pragma unroll
      for (int q = 0; q < NW; ++q)
#pragma unroll
        for (int t = 0; t < MT; ++t) acc[q][t] = M::mma(af[0][u][t], wf[0][u][q], acc[q][t]);
    if (s + kU < s1) {
      if (s + 2 * kU < s1) load(0, s + 2 * kU);
#pragma unroll
      for (int u = 0; u < kU; ++u)
#pragma unroll
        for (int q = 0; q < NW; ++q)
#pragma unroll
          for (int t = 0; t < MT; ++t) acc[q][t] = M::mma(af[1][u][t], wf[1][u][q], acc[q][t]);
    }
  }
#pragma unroll
  for (int q = 0; q < NW; ++q)
#pragma unroll
    for (int t = 0; t < MT; ++t)
#pragma unroll
      for (int i = 0; i < 4; ++i) red[wave][4 * (q * MT + t) + i][lane] = acc[q][t][i];
  __syncthreads();
  const int ti = threadIdx.x >> 6;  // 4 t + i, one per wave
  if (ti >= 4 * MT) return;
  const int m = 16 * (ti >> 2) + 4 * g + (ti & 3), n = n0 + r;
  float v = 0.f;
#pragma unroll
  for (int w = 0; w < kWaves; ++w) v += red[w][ti][lane];
  const bool ok = m < p.M && n < p.N;
  const float rs = p.ssq_in ? rstd[min(m, p.M - 1)] : 1.f;
  v *= rs;
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
  if constexpr (EPI == kGeglu) {
    float up = 0.f;
#pragma unroll
    for (int w = 0; w < kWaves; ++w) up += red[w][4 * MT + ti][lane];
    v = gelu_tanh(v) * (up * rs);
  }
  if constexpr (EPI == kCap) {
    if (ok) p.yf[at] = p.cap * tanhf(v / p.cap);
    return;
  }
  if constexpr (EPI == kStream || EPI == kPost) {
    float sq = 0.f;
    if (ok) {
      float x = p.x[at];
      if constexpr (EPI == kPost) {
        if (p.res_ssq) x *= rres[m] * bf2f(p.res_w[n]);
        x = p.alpha * x + v;
        if (p.bias) x += bf2f(p.bias[n]);
      } else {
        x += v;
      }
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
  else if (epi == kStream) stream_gemm_kernel<MT, kStream><<<g, 64 * kWaves, 0, st>>>(p);
  else if (epi == kPost) stream_gemm_kernel<MT, kPost><<<g, 64 * kWaves, 0, st>>>(p);
  else if (epi == kGeglu) stream_gemm_kernel<MT, kGeglu><<<g, 64 * kWaves, 0, st>>>(p);
  else stream_gemm_kernel<MT, kCap><<<g, 64 * kWaves, 0, st>>>(p);
}

}  // namespace

void launch_stream_gemm(const StreamGemmParams& p, int epi, hipStream_t st) {
  if (p.M <= 16) go<1>(p, epi, st);
  else go<2>(p, epi, st);
}

}  // namespace dla
