// Attention inside chunks of the sequence for gfx950: position i sees the positions j <= i with
// floor(j / chunk) = floor(i / chunk).
//
//   prepare   biases, RMS norms of q and k over their whole projections, rotation of each head's first
//             `rot` dimensions, values as projected; prompts write q / k / v, decode writes k and v
//             straight into the cache
//   store     the last chunk's keys and values of a portion into the cache (after its attention: the
//             portion's first queries may still need what these rows replace)
//   prefill   any head sizes, bf16 or fp32 (bf16 sizes of chunk_prefill.hip take that kernel)
//   decode    split keys (bf16 sizes of chunk_decode.hip take that kernel)
//   combine   merge of the splits
//
// Cache rows are [B, G, rows, .]: position p sits in row p % chunk. A token's position is its column minus
// kv_start[b]; columns below that are padding, never seen as keys. Scores, weights and sums are fp32.
#include "mix_params.h"
#include "mma.h"

namespace dla {

bool chunk_decode_mfma_ok(const ChunkAttnParams&);  // chunk_decode.hip
void launch_chunk_decode_mfma(const ChunkAttnParams&, hipStream_t);

namespace {

constexpr float kLog2e = 1.4426950408889634f;

// ------------------------------------------------------------------------------------ prepare
// one workgroup per token
template <typename T, int VEC, bool DECODE>
__global__ __launch_bounds__(256) void chunk_prepare_kernel(ChunkAttnParams p) {
  __shared__ float scratch[4];
  const int64_t rowi = blockIdx.x;
  const int b = static_cast<int>(rowi / p.T), t = static_cast<int>(rowi % p.T);
  const int nq = p.H * p.dim, nk = p.G * p.dim, nv = p.G * p.vdim, half = p.rot >> 1;
  const T *in = static_cast<const T*>(p.row) + rowi * p.ld, *bias = static_cast<const T*>(p.bias);
  float sq = 0.f, sk = 0.f, v[VEC], w[VEC];
  for (int i = threadIdx.x * VEC; i < nq + nk; i += 256 * VEC) {
    load_vec<T, VEC>(in + i, v);
    load_vec<T, VEC>(bias + i, w);
    float s = 0.f;
#pragma unroll
    for (int e = 0; e < VEC; ++e) s += (v[e] + w[e]) * (v[e] + w[e]);
    if (i < nq) sq += s;  // (VEC divides nq: a vector never straddles)
    else sk += s;
  }
  const float rq = rsqrtf(block_sum<256>(sq, scratch) / nq + p.eps);
  const float rk = rsqrtf(block_sum<256>(sk, scratch) / nk + p.eps);
  const int64_t pos = max((DECODE ? p.slot[0] : p.base) + t - (p.kv_start ? p.kv_start[b] : 0), static_cast<int64_t>(0));
  const int64_t pt = min(pos, static_cast<int64_t>(max(p.npos - 1, 0)));
  const float *cs = p.cos_t + pt * half, *sn = p.sin_t + pt * half;
  const int64_t crow = min(pos % p.chunk, static_cast<int64_t>(p.rows - 1));  // (a full cache is the host's error)
  for (int i = threadIdx.x * VEC; i < nq + nk; i += 256 * VEC) {
    const bool is_k = i >= nq;
    const int j = is_k ? i - nq : i, d = j % p.dim, hd = j / p.dim;
    const T* nw = static_cast<const T*>(is_k ? p.k_w : p.q_w);
    const float r = is_k ? rk : rq;
    auto normed = [&](int off, float* o) {  // VEC normed values `off` away, before rotation
      float x[VEC], y[VEC], z[VEC];
      load_vec<T, VEC>(in + i + off, x);
      load_vec<T, VEC>(bias + i + off, y);
      load_vec<T, VEC>(nw + j + off, z);
#pragma unroll
      for (int e = 0; e < VEC; ++e) o[e] = (x[e] + y[e]) * r * z[e];
    };
    normed(0, v);
    if (d < p.rot) {
      const bool lo = d < half;
      normed(lo ? half : -half, w);
      const int c = lo ? d : d - half;
#pragma unroll
      for (int e = 0; e < VEC; ++e) v[e] = lo ? v[e] * cs[c + e] - w[e] * sn[c + e] : v[e] * cs[c + e] + w[e] * sn[c + e];
    }
    T* out;
    if (!is_k) out = static_cast<T*>(p.q) + rowi * nq + j;
    else if (DECODE) out = static_cast<T*>(p.kc) + ((static_cast<int64_t>(b) * p.G + hd) * p.rows + crow) * p.dim + d;
    else out = static_cast<T*>(p.k) + rowi * nk + j;
    store_vec<T, VEC>(out, v);
  }
  for (int i = threadIdx.x * VEC; i < nv; i += 256 * VEC) {
    load_vec<T, VEC>(in + p.v_off + i, v);
    load_vec<T, VEC>(bias + p.v_off + i, w);
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] += w[e];
    T* out = DECODE ? static_cast<T*>(p.vc) + ((static_cast<int64_t>(b) * p.G + i / p.vdim) * p.rows + crow) * p.vdim + i % p.vdim
                    : static_cast<T*>(p.v) + rowi * nv + i;
    store_vec<T, VEC>(out, v);
  }
}

// -------------------------------------------------------------------------------------- store
// grid (ceil(min(T, chunk) / 16), G, B), 256 threads, 16 lanes per token: the n-th last token, if it belongs to
// the last token's chunk
template <typename T, int VEC>
__global__ __launch_bounds__(256) void chunk_store_kernel(ChunkAttnParams p) {
  const int b = blockIdx.z, hd = blockIdx.y, n = blockIdx.x * 16 + (threadIdx.x >> 4), t = p.T - 1 - n;
  const int64_t last = p.base + p.T - 1 - (p.kv_start ? p.kv_start[b] : 0), pos = last - n;
  if (t < 0 || pos < 0 || static_cast<int64_t>(n) > last % p.chunk) return;
  const int64_t crow = pos % p.chunk, g = static_cast<int64_t>(b) * p.T + t, c = (static_cast<int64_t>(b) * p.G + hd) * p.rows + crow;
  if (crow >= p.rows) return;
  float v[VEC];
  for (int i = (threadIdx.x & 15) * VEC; i < p.dim; i += 16 * VEC) {
    load_vec<T, VEC>(static_cast<const T*>(p.k) + (g * p.G + hd) * p.dim + i, v);
    store_vec<T, VEC>(static_cast<T*>(p.kc) + c * p.dim + i, v);
  }
  for (int i = (threadIdx.x & 15) * VEC; i < p.vdim; i += 16 * VEC) {
    load_vec<T, VEC>(static_cast<const T*>(p.v) + (g * p.G + hd) * p.vdim + i, v);
    store_vec<T, VEC>(static_cast<T*>(p.vc) + c * p.vdim + i, v);
  }
}

// ----------------------------------------------------------------- any sizes: one query per wave
// Keys of one query in tiles of 64: a lane per key for the score, a lane per value column (and 64
// more, ...) for the weighted sum. qs: the query in LDS; key / value rows by position through `kv`.
template <typename T, typename F>
__device__ __forceinline__ void one_query(const ChunkAttnParams& p, const float* qs, int64_t lo, int64_t hi, float* os, F kv,
                                          float& m_run, float& l_run) {
  const int lane = threadIdx.x & 63;
  const float c = p.scale * kLog2e;
  m_run = -INFINITY;
  l_run = 0.f;
  __builtin_amdgcn_wave_barrier();  // (one wave: its LDS accesses stay in order)
  for (int v = lane; v < p.vdim; v += 64) os[v] = 0.f;
  for (int64_t j0 = lo; j0 < hi; j0 += 64) {
    const int cnt = static_cast<int>(min(hi - j0, static_cast<int64_t>(64)));
    float s = -INFINITY;
    if (lane < cnt) {
      const T *kr, *vr;
      kv(j0 + lane, kr, vr);
      s = 0.f;
      for (int d = 0; d < p.dim; ++d) s += qs[d] * to_f<T>(kr[d]);
      s *= c;
    }
    const float mn = fmaxf(m_run, wave_max(s)), a = exp2f(m_run - mn), e = exp2f(s - mn);  // (cnt >= 1: mn is finite)
    m_run = mn;
    l_run = l_run * a + wave_sum(e);
    for (int v0 = 0; v0 < p.vdim; v0 += 64) {
      const int v = v0 + lane;
      float o = v < p.vdim ? os[v] * a : 0.f;
      for (int n = 0; n < cnt; ++n) {
        const float w = __shfl(e, n, 64);
        const T *kr, *vr;
        kv(j0 + n, kr, vr);
        if (v < p.vdim) o += w * to_f<T>(vr[v]);
      }
      if (v < p.vdim) os[v] = o;
    }
  }
}

// grid (ceil(T / 4), H, B), 4 waves, one query each
template <typename T>
__global__ __launch_bounds__(256) void chunk_prefill_any_kernel(ChunkAttnParams p) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, h = blockIdx.y, b = blockIdx.z;
  const int t = blockIdx.x * 4 + wave, hk = h / (p.H / p.G);
  float* qs = reinterpret_cast<float*>(smem) + wave * (p.dim + p.vdim);
  float* os = qs + p.dim;
  if (t >= p.T) return;  // (no barrier below)
  const int64_t row = static_cast<int64_t>(b) * p.T + t, off = p.base - (p.kv_start ? p.kv_start[b] : 0), pos = off + t;
  T* O = static_cast<T*>(p.o) + (row * p.H + h) * p.vdim;
  for (int d = lane; d < p.dim; d += 64) qs[d] = to_f<T>(static_cast<const T*>(p.q)[(row * p.H + h) * p.dim + d]);
  const int64_t first = pos < 0 ? 0 : pos - pos % p.chunk;
  float m, l;
  one_query<T>(p, qs, first, pos + 1, os, [&](int64_t j, const T*& kr, const T*& vr) {
    if (j >= off) {
      const int64_t g = (static_cast<int64_t>(b) * p.T + (j - off)) * p.G + hk;
      kr = static_cast<const T*>(p.k) + g * p.dim;
      vr = static_cast<const T*>(p.v) + g * p.vdim;
    } else {
      const int64_t g = (static_cast<int64_t>(b) * p.G + hk) * p.rows + j % p.chunk;
      kr = static_cast<const T*>(p.kc) + g * p.dim;
      vr = static_cast<const T*>(p.vc) + g * p.vdim;
    }
  }, m, l);
  for (int v = lane; v < p.vdim; v += 64) O[v] = from_f<T>(l > 0.f ? os[v] / l : 0.f);
}

// grid (ns, H, B), one wave
template <typename T>
__global__ __launch_bounds__(64) void chunk_decode_any_kernel(ChunkAttnParams p) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  const int lane = threadIdx.x, h = blockIdx.y, b = blockIdx.z, hk = h / (p.H / p.G);
  float* qs = reinterpret_cast<float*>(smem);
  float* os = qs + p.dim;
  const int64_t bh = static_cast<int64_t>(b) * p.H + h;
  for (int d = lane; d < p.dim; d += 64) qs[d] = to_f<T>(static_cast<const T*>(p.q)[bh * p.dim + d]);
  const int64_t pos = max(p.slot[0] - (p.kv_start ? p.kv_start[b] : 0), static_cast<int64_t>(0));
  const int64_t n = min(pos % p.chunk + 1, static_cast<int64_t>(p.rows)), per = (n + p.ns - 1) / p.ns;
  const int64_t k0 = blockIdx.x * per, k1 = min(k0 + per, n);
  const int64_t base = (static_cast<int64_t>(b) * p.G + hk) * p.rows;
  float m, l;
  one_query<T>(p, qs, k0, k1, os, [&](int64_t j, const T*& kr, const T*& vr) {
    kr = static_cast<const T*>(p.kc) + (base + j) * p.dim;
    vr = static_cast<const T*>(p.vc) + (base + j) * p.vdim;
  }, m, l);
  if (p.ns == 1) {
    for (int v = lane; v < p.vdim; v += 64) static_cast<T*>(p.o)[bh * p.vdim + v] = from_f<T>(os[v] / l);
    return;
  }
  const int64_t at = bh * p.ns + blockIdx.x;
  for (int v = lane; v < p.vdim; v += 64) p.part_o[at * p.vdim + v] = os[v];
  if (lane == 0) {
    p.part_ml[2 * at] = m;
    p.part_ml[2 * at + 1] = l;
  }
}

// grid (H, B), 256 threads: o = sum_s 2^(m_s - m) o_s / sum_s 2^(m_s - m) l_s (ns <= 256)
template <typename T>
__global__ __launch_bounds__(256) void chunk_combine_kernel(ChunkAttnParams p) {
  __shared__ float scratch[4], ws[256];
  const int64_t bh = static_cast<int64_t>(blockIdx.y) * p.H + blockIdx.x;
  const bool in = static_cast<int>(threadIdx.x) < p.ns;
  const float m = in ? p.part_ml[2 * (bh * p.ns + threadIdx.x)] : -INFINITY;
  const float l = in ? p.part_ml[2 * (bh * p.ns + threadIdx.x) + 1] : 0.f;
  const float mx = block_max<256>(m, scratch);
  const float w = m == -INFINITY ? 0.f : exp2f(m - mx);
  const float total = block_sum<256>(w * l, scratch);
  ws[threadIdx.x] = w;
  __syncthreads();
  for (int v = threadIdx.x; v < p.vdim; v += 256) {
    float o = 0.f;
    for (int s = 0; s < p.ns; ++s)
      if (ws[s] != 0.f) o += ws[s] * p.part_o[(bh * p.ns + s) * p.vdim + v];
    static_cast<T*>(p.o)[bh * p.vdim + v] = from_f<T>(o / total);
  }
}

template <typename T>
bool vec_ok(const ChunkAttnParams& p) {
  const auto al = [](const void* x) { return reinterpret_cast<uintptr_t>(x) % 16 == 0; };
  return p.dim % 8 == 0 && p.vdim % 8 == 0 && p.rot % 16 == 0 && p.ld % 8 == 0 && p.v_off % 8 == 0 && al(p.row) && al(p.bias) &&
         al(p.q_w) && al(p.k_w) && al(p.q) && al(p.k) && al(p.v) && al(p.kc) && al(p.vc);
}

template <typename T>
void prepare(const ChunkAttnParams& p, bool decode, hipStream_t st) {
  const dim3 g(static_cast<unsigned>(static_cast<int64_t>(p.B) * p.T));
  const bool v = vec_ok<T>(p);
  if (decode) {
    if (v) chunk_prepare_kernel<T, 8, true><<<g, 256, 0, st>>>(p);
    else chunk_prepare_kernel<T, 1, true><<<g, 256, 0, st>>>(p);
  } else {
    if (v) chunk_prepare_kernel<T, 8, false><<<g, 256, 0, st>>>(p);
    else chunk_prepare_kernel<T, 1, false><<<g, 256, 0, st>>>(p);
  }
}

template <typename T>
void store(const ChunkAttnParams& p, hipStream_t st) {
  const dim3 g(((p.T < p.chunk ? p.T : p.chunk) + 15) / 16, p.G, p.B);
  const auto al = [](const void* x) { return reinterpret_cast<uintptr_t>(x) % 16 == 0; };
  if (p.dim % 8 == 0 && p.vdim % 8 == 0 && al(p.k) && al(p.v) && al(p.kc) && al(p.vc)) chunk_store_kernel<T, 8><<<g, 256, 0, st>>>(p);
  else chunk_store_kernel<T, 1><<<g, 256, 0, st>>>(p);
}

}  // namespace

void launch_chunk_prepare(bool bf16, const ChunkAttnParams& p, bool decode, hipStream_t st) {
  if (bf16) prepare<bf16_t>(p, decode, st);
  else prepare<float>(p, decode, st);
}

void launch_chunk_store(bool bf16, const ChunkAttnParams& p, hipStream_t st) {
  if (bf16) store<bf16_t>(p, st);
  else store<float>(p, st);
}

void launch_chunk_prefill_any(bool bf16, const ChunkAttnParams& p, hipStream_t st) {
  const dim3 g((p.T + 3) / 4, p.H, p.B);
  const int lds = 16 * (p.dim + p.vdim);
  if (bf16) chunk_prefill_any_kernel<bf16_t><<<g, 256, lds, st>>>(p);
  else chunk_prefill_any_kernel<float><<<g, 256, lds, st>>>(p);
}

// attention over the cache and, if the keys were split, the merge
void launch_chunk_decode(bool bf16, const ChunkAttnParams& p, hipStream_t st) {
  if (bf16 && chunk_decode_mfma_ok(p)) {
    launch_chunk_decode_mfma(p, st);
  } else {
    const dim3 g(p.ns, p.H, p.B);
    const int lds = 4 * (p.dim + p.vdim);
    if (bf16) chunk_decode_any_kernel<bf16_t><<<g, 64, lds, st>>>(p);
    else chunk_decode_any_kernel<float><<<g, 64, lds, st>>>(p);
  }
  if (p.ns > 1) {
    if (bf16) chunk_combine_kernel<bf16_t><<<dim3(p.H, p.B), 256, 0, st>>>(p);
    else chunk_combine_kernel<float><<<dim3(p.H, p.B), 256, 0, st>>>(p);
  }
}

}  // namespace dla
