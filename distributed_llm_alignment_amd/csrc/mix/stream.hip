// Kernels on the fp32 residual stream of per-layer designs: scaled embedding, the stream update +
// RMS norm, the norm after a sum, the per-layer token input's gate, squared ReLU, gelu-gated units,
// the soft cap of the logits.
#include "mma.h"

namespace dla {
namespace {

template <typename T>
__global__ __launch_bounds__(256) void embed_stream_kernel(const int64_t* __restrict__ ids, const T* __restrict__ table,
                                                           float scale, float* __restrict__ out, int* __restrict__ bad,
                                                           int64_t V, int H) {
  const int64_t row = blockIdx.x;
  const int64_t id = ids[row];
  const bool ok = id >= 0 && id < V;
  if (!ok && threadIdx.x == 0) bad[0] = 1;
  const T* src = table + (ok ? id : 0) * H;
  const float f = ok ? scale : 0.f;
  if (H % 4 == 0) {
    for (int c = 4 * threadIdx.x; c < H; c += 4 * blockDim.x) {
      float v[4];
      load_vec<T, 4>(src + c, v);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = ok ? v[e] * f : 0.f;
      store_vec<float, 4>(out + row * H + c, v);
    }
  } else {
    for (int c = threadIdx.x; c < H; c += blockDim.x) out[row * H + c] = ok ? to_f<T>(src[c]) * f : 0.f;
  }
}

template <int NT>
__device__ __forceinline__ float row_sum(float v, float* scratch) {
  if constexpr (NT == 64) return wave_sum(v);
  return block_sum<NT>(v, scratch);
}

// One row per workgroup, kept in registers (H % 4 == 0, H <= 4 * NT * NV).
//   x += delta                       (DW: RMSNorm(delta) * delta_w)
//   x += inject
//   y = RMSNorm(x) * (offset + w)    (w == nullptr: y = x)
template <typename T, int NT, int NV>
__global__ __launch_bounds__(NT) void stream_norm_kernel(float* __restrict__ x, const T* __restrict__ delta,
                                                         const T* __restrict__ delta_w, const float* __restrict__ inject,
                                                         const T* __restrict__ w, T* __restrict__ y, float eps,
                                                         float offset, int H) {
  __shared__ float scratch[NT / 64];
  const int64_t base = static_cast<int64_t>(blockIdx.x) * H;
  float xv[NV][4], dv[NV][4];
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = 4 * (threadIdx.x + NT * j);
    if (c < H) load_vec<float, 4>(x + base + c, xv[j]);
#pragma unroll
    for (int e = 0; e < 4; ++e) dv[j][e] = 0.f;
    if (c < H && delta) load_vec<T, 4>(delta + base + c, dv[j]);
  }
  float wv[NV][4], iv[NV][4];
#pragma unroll
  for (int j = 0; j < NV; ++j) {  // (in flight behind the sums)
    const int c = 4 * (threadIdx.x + NT * j);
    if (c < H && w) load_vec<T, 4>(w + c, wv[j]);
#pragma unroll
    for (int e = 0; e < 4; ++e) iv[j][e] = 0.f;
    if (c < H && inject) load_vec<float, 4>(inject + base + c, iv[j]);
  }
  if (delta_w) {
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < NV; ++j)
#pragma unroll
      for (int e = 0; e < 4; ++e) ss += dv[j][e] * dv[j][e];
    const float r = rsqrtf(row_sum<NT>(ss, scratch) / H + eps);
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int c = 4 * (threadIdx.x + NT * j);
      if (c < H) {
        float dw[4];
        load_vec<T, 4>(delta_w + c, dw);
#pragma unroll
        for (int e = 0; e < 4; ++e) dv[j][e] *= r * dw[e];
      }
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = 4 * (threadIdx.x + NT * j);
    if (c >= H) continue;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      xv[j][e] = xv[j][e] + dv[j][e] + iv[j][e];
      ss += xv[j][e] * xv[j][e];
    }
    if (delta || inject) store_vec<float, 4>(x + base + c, xv[j]);
  }
  const float r = w ? rsqrtf(row_sum<NT>(ss, scratch) / H + eps) : 1.f;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = 4 * (threadIdx.x + NT * j);
    if (c >= H) continue;
    float yv[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) yv[e] = w ? xv[j][e] * r * (offset + wv[j][e]) : xv[j][e];
    store_vec<T, 4>(y + base + c, yv);
  }
}

// Any H: the row is read again from memory instead of kept (each thread re-reads its own elements).
template <typename T>
__global__ __launch_bounds__(256) void stream_norm_any_kernel(float* __restrict__ x, const T* __restrict__ delta,
                                                              const T* __restrict__ delta_w,
                                                              const float* __restrict__ inject, const T* __restrict__ w,
                                                              T* __restrict__ y, float eps, float offset, int H) {
  __shared__ float scratch[4];
  const int64_t base = static_cast<int64_t>(blockIdx.x) * H;
  float dr = 1.f;
  if (delta_w) {
    float ss = 0.f;
    for (int c = threadIdx.x; c < H; c += 256) {
      const float d = to_f<T>(delta[base + c]);
      ss += d * d;
    }
    dr = rsqrtf(block_sum<256>(ss, scratch) / H + eps);
  }
  float ss = 0.f;
  for (int c = threadIdx.x; c < H; c += 256) {
    float v = x[base + c];
    if (delta) v += delta_w ? to_f<T>(delta[base + c]) * (dr * to_f<T>(delta_w[c])) : to_f<T>(delta[base + c]);
    if (inject) v += inject[base + c];
    ss += v * v;
    if (delta || inject) x[base + c] = v;
  }
  const float r = w ? rsqrtf(block_sum<256>(ss, scratch) / H + eps) : 1.f;
  for (int c = threadIdx.x; c < H; c += 256) {
    const float v = x[base + c];
    y[base + c] = from_f<T>(w ? v * r * (offset + to_f<T>(w[c])) : v);
  }
}

// One row per workgroup, kept in registers (H % 4 == 0, H <= 4 * NT * NV).
//   x <- RMSNorm(alpha x + delta + bias) * w
//   y = x, or RMSNorm(x) * w2
template <typename T, int NT, int NV>
__global__ __launch_bounds__(NT) void post_norm_kernel(float* __restrict__ x, const T* __restrict__ delta,
                                                       const T* __restrict__ bias, float alpha, const T* __restrict__ w,
                                                       const T* __restrict__ w2, T* __restrict__ y, float eps, int H) {
  __shared__ float scratch[NT / 64];
  const int64_t base = static_cast<int64_t>(blockIdx.x) * H;
  float xv[NV][4], wv[NV][4], w2v[NV][4], ss = 0.f;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = 4 * (threadIdx.x + NT * j);
    float dv[4] = {0.f, 0.f, 0.f, 0.f}, bv[4] = {0.f, 0.f, 0.f, 0.f};
    if (c < H) {
      load_vec<float, 4>(x + base + c, xv[j]);
      if (delta) load_vec<T, 4>(delta + base + c, dv);
      if (bias) load_vec<T, 4>(bias + c, bv);
      load_vec<T, 4>(w + c, wv[j]);
      if (w2) load_vec<T, 4>(w2 + c, w2v[j]);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        xv[j][e] = alpha * xv[j][e] + dv[e] + bv[e];
        ss += xv[j][e] * xv[j][e];
      }
    }
  }
  const float r = rsqrtf(row_sum<NT>(ss, scratch) / H + eps);
  ss = 0.f;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = 4 * (threadIdx.x + NT * j);
    if (c >= H) continue;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      xv[j][e] = xv[j][e] * r * wv[j][e];
      ss += xv[j][e] * xv[j][e];
    }
    store_vec<float, 4>(x + base + c, xv[j]);
  }
  const float r2 = w2 ? rsqrtf(row_sum<NT>(ss, scratch) / H + eps) : 1.f;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = 4 * (threadIdx.x + NT * j);
    if (c >= H) continue;
    if (w2) {
#pragma unroll
      for (int e = 0; e < 4; ++e) xv[j][e] = xv[j][e] * r2 * w2v[j][e];
    }
    store_vec<T, 4>(y + base + c, xv[j]);
  }
}

// Any H: every thread re-reads its own elements.
template <typename T>
__global__ __launch_bounds__(256) void post_norm_any_kernel(float* __restrict__ x, const T* __restrict__ delta,
                                                            const T* __restrict__ bias, float alpha,
                                                            const T* __restrict__ w, const T* __restrict__ w2,
                                                            T* __restrict__ y, float eps, int H) {
  __shared__ float scratch[4];
  const int64_t base = static_cast<int64_t>(blockIdx.x) * H;
  float ss = 0.f;
  for (int c = threadIdx.x; c < H; c += 256) {
    const float v = alpha * x[base + c] + (delta ? to_f<T>(delta[base + c]) : 0.f) + (bias ? to_f<T>(bias[c]) : 0.f);
    ss += v * v;
    x[base + c] = v;
  }
  const float r = rsqrtf(block_sum<256>(ss, scratch) / H + eps);
  ss = 0.f;
  for (int c = threadIdx.x; c < H; c += 256) {
    const float v = x[base + c] * r * to_f<T>(w[c]);
    ss += v * v;
    x[base + c] = v;
  }
  const float r2 = w2 ? rsqrtf(block_sum<256>(ss, scratch) / H + eps) : 1.f;
  for (int c = threadIdx.x; c < H; c += 256)
    y[base + c] = from_f<T>(w2 ? x[base + c] * r2 * to_f<T>(w2[c]) : x[base + c]);
}

// one wave per row
template <typename T, int VEC>
__global__ __launch_bounds__(256) void side_gate_kernel(const T* __restrict__ z, const int64_t* __restrict__ ids,
                                                        const T* __restrict__ table, int64_t ldt, int64_t off,
                                                        T* __restrict__ out, int64_t rows, int dim, int64_t V) {
  const int64_t row = blockIdx.x * 4ll + (threadIdx.x >> 6);
  if (row >= rows) return;
  const int64_t id = ids[row];
  const bool ok = id >= 0 && id < V;
  for (int c = (threadIdx.x & 63) * VEC; c < dim; c += 64 * VEC) {
    float v[VEC], e[VEC];
    load_vec<T, VEC>(z + row * dim + c, v);
    load_vec<T, VEC>(table + (ok ? id : 0) * ldt + off + c, e);
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[j] = ok ? gelu_tanh(v[j]) * e[j] : 0.f;
    store_vec<T, VEC>(out + row * dim + c, v);
  }
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void relu2_kernel(const T* __restrict__ u, T* __restrict__ y, int64_t n) {
  for (int64_t i = (blockIdx.x * 256ll + threadIdx.x) * VEC; i < n; i += gridDim.x * 256ll * VEC) {
    float v[VEC];
    load_vec<T, VEC>(u + i, v);
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      const float r = fmaxf(v[e], 0.f);
      v[e] = r * r;
    }
    store_vec<T, VEC>(y + i, v);
  }
}

// u [rows, 2 F] = [gate | up] -> gelu_tanh(gate) * up; n = rows * F / VEC
template <typename T, int VEC>
__global__ __launch_bounds__(256) void geglu_kernel(const T* __restrict__ u, T* __restrict__ y, int64_t n, int F) {
  const int fv = F / VEC;
  for (int64_t i = blockIdx.x * 256ll + threadIdx.x; i < n; i += gridDim.x * 256ll) {
    const int64_t row = i / fv;
    const int c = static_cast<int>(i - row * fv) * VEC;
    float a[VEC], b[VEC];
    load_vec<T, VEC>(u + row * 2 * F + c, a);
    load_vec<T, VEC>(u + row * 2 * F + F + c, b);
#pragma unroll
    for (int e = 0; e < VEC; ++e) a[e] = gelu_tanh(a[e]) * b[e];
    store_vec<T, VEC>(y + row * F + c, a);
  }
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void softcap_kernel(const T* __restrict__ z, float* __restrict__ y, int64_t n, float cap) {
  const float inv = 1.f / cap;
  for (int64_t i = (blockIdx.x * 256ll + threadIdx.x) * VEC; i < n; i += gridDim.x * 256ll * VEC) {
    float v[VEC];
    load_vec<T, VEC>(z + i, v);
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = cap * tanhf(v[e] * inv);
    store_vec<float, VEC>(y + i, v);
  }
}

inline unsigned grid_for(int64_t work) {
  const int64_t b = (work + 255) / 256;
  return static_cast<unsigned>(b < 1 ? 1 : (b > 8192 ? 8192 : b));
}

template <typename T>
void norm_dispatch(float* x, const T* delta, const T* dw, const float* inject, const T* w, T* y, float eps,
                   float offset, int64_t rows, int H, hipStream_t st) {
  const dim3 g(static_cast<unsigned>(rows));
#define DLA_NORM(NT, NV) stream_norm_kernel<T, NT, NV><<<g, NT, 0, st>>>(x, delta, dw, inject, w, y, eps, offset, H)
  const auto al = [](const void* q) { return reinterpret_cast<uintptr_t>(q) % 8 == 0; };
  if (H % 4 || H > 16384 || !al(delta) || !al(dw) || !al(w) || !al(y)) stream_norm_any_kernel<T><<<g, 256, 0, st>>>(x, delta, dw, inject, w, y, eps, offset, H);
  else if (H <= 256) DLA_NORM(64, 1);
  else if (rows <= 64 && H > 2048) {  // decode: short latency chain
    if (H <= 4096) DLA_NORM(1024, 1);
    else if (H <= 8192) DLA_NORM(1024, 2);
    else DLA_NORM(1024, 4);
  } else if (rows <= 64 && H > 1024) DLA_NORM(512, 1);
  else if (H <= 1024) DLA_NORM(256, 1);
  else if (H <= 2048) DLA_NORM(256, 2);
  else if (H <= 4096) DLA_NORM(256, 4);
  else if (H <= 8192) DLA_NORM(256, 8);
  else DLA_NORM(1024, 4);
#undef DLA_NORM
}

template <typename T>
void post_dispatch(float* x, const T* delta, const T* bias, float alpha, const T* w, const T* w2, T* y, float eps,
                   int64_t rows, int H, hipStream_t st) {
  const dim3 g(static_cast<unsigned>(rows));
#define DLA_POST(NT, NV) post_norm_kernel<T, NT, NV><<<g, NT, 0, st>>>(x, delta, bias, alpha, w, w2, y, eps, H)
  const auto al = [](const void* q) { return reinterpret_cast<uintptr_t>(q) % 16 == 0; };
  if (H % 4 || H > 16384 || !al(delta) || !al(bias) || !al(w) || !al(w2) || !al(y))
    post_norm_any_kernel<T><<<g, 256, 0, st>>>(x, delta, bias, alpha, w, w2, y, eps, H);
  else if (H <= 256) DLA_POST(64, 1);
  else if (rows <= 64 && H > 2048) {  // decode: short latency chain
    if (H <= 4096) DLA_POST(1024, 1);
    else if (H <= 8192) DLA_POST(1024, 2);
    else DLA_POST(1024, 4);
  } else if (rows <= 64 && H > 1024) DLA_POST(512, 1);
  else if (H <= 1024) DLA_POST(256, 1);
  else if (H <= 2048) DLA_POST(256, 2);
  else if (H <= 4096) DLA_POST(256, 4);
  else if (H <= 8192) DLA_POST(256, 8);
  else DLA_POST(1024, 4);
#undef DLA_POST
}

}  // namespace

void launch_post_norm(bool bf16, float* x, const void* delta, const void* bias, float alpha, const void* w, const void* w2,
                      void* y, float eps, int64_t rows, int H, hipStream_t st) {
  if (rows == 0) return;
  if (bf16)
    post_dispatch<bf16_t>(x, static_cast<const bf16_t*>(delta), static_cast<const bf16_t*>(bias), alpha,
                          static_cast<const bf16_t*>(w), static_cast<const bf16_t*>(w2), static_cast<bf16_t*>(y), eps, rows,
                          H, st);
  else
    post_dispatch<float>(x, static_cast<const float*>(delta), static_cast<const float*>(bias), alpha,
                         static_cast<const float*>(w), static_cast<const float*>(w2), static_cast<float*>(y), eps, rows, H,
                         st);
}

void launch_geglu(bool bf16, const void* u, void* y, int64_t rows, int F, hipStream_t st) {
  if (rows == 0) return;
  const bool vec = F % 8 == 0 && reinterpret_cast<uintptr_t>(u) % 16 == 0 && reinterpret_cast<uintptr_t>(y) % 16 == 0;
  const int64_t n = rows * (vec ? F / 8 : F);
#define DLA_GEGLU(T, V) geglu_kernel<T, V><<<grid_for(n), 256, 0, st>>>(static_cast<const T*>(u), static_cast<T*>(y), n, F)
  if (bf16) {
    if (vec) DLA_GEGLU(bf16_t, 8);
    else DLA_GEGLU(bf16_t, 1);
  } else {
    if (vec) DLA_GEGLU(float, 8);
    else DLA_GEGLU(float, 1);
  }
#undef DLA_GEGLU
}

void launch_softcap(bool bf16, const void* z, float* y, int64_t n, float cap, hipStream_t st) {
  if (n == 0) return;
  const bool vec = n % 4 == 0 && reinterpret_cast<uintptr_t>(z) % 16 == 0;
#define DLA_CAP(T, V) softcap_kernel<T, V><<<grid_for(n / V), 256, 0, st>>>(static_cast<const T*>(z), y, n, cap)
  if (bf16) {
    if (vec) DLA_CAP(bf16_t, 4);
    else DLA_CAP(bf16_t, 1);
  } else {
    if (vec) DLA_CAP(float, 4);
    else DLA_CAP(float, 1);
  }
#undef DLA_CAP
}

void launch_embed_stream(bool bf16, const int64_t* ids, const void* table, float scale, float* out, int* bad,
                         int64_t rows, int64_t V, int H, hipStream_t st) {
  if (rows == 0) return;
  const dim3 g(static_cast<unsigned>(rows));
  if (bf16) embed_stream_kernel<bf16_t><<<g, 256, 0, st>>>(ids, static_cast<const bf16_t*>(table), scale, out, bad, V, H);
  else embed_stream_kernel<float><<<g, 256, 0, st>>>(ids, static_cast<const float*>(table), scale, out, bad, V, H);
}

void launch_stream_norm(bool bf16, float* x, const void* delta, const void* dw, const float* inject, const void* w,
                        void* y, float eps, float offset, int64_t rows, int H, hipStream_t st) {
  if (rows == 0) return;
  if (bf16)
    norm_dispatch<bf16_t>(x, static_cast<const bf16_t*>(delta), static_cast<const bf16_t*>(dw), inject,
                          static_cast<const bf16_t*>(w), static_cast<bf16_t*>(y), eps, offset, rows, H, st);
  else
    norm_dispatch<float>(x, static_cast<const float*>(delta), static_cast<const float*>(dw), inject,
                         static_cast<const float*>(w), static_cast<float*>(y), eps, offset, rows, H, st);
}

void launch_side_gate(bool bf16, const void* z, const int64_t* ids, const void* table, int64_t ldt, int64_t off,
                      void* out, int64_t rows, int dim, int64_t V, hipStream_t st) {
  if (rows == 0) return;
  const dim3 g(static_cast<unsigned>((rows + 3) / 4));
  const bool vec = dim % 4 == 0 && ldt % 4 == 0 && off % 4 == 0 &&
                   (reinterpret_cast<uintptr_t>(z) | reinterpret_cast<uintptr_t>(table) | reinterpret_cast<uintptr_t>(out)) % 16 == 0;
#define DLA_GATE(T, V4) \
  side_gate_kernel<T, V4><<<g, 256, 0, st>>>(static_cast<const T*>(z), ids, static_cast<const T*>(table), ldt, off, static_cast<T*>(out), rows, dim, V)
  if (bf16) {
    if (vec) DLA_GATE(bf16_t, 4);
    else DLA_GATE(bf16_t, 1);
  } else {
    if (vec) DLA_GATE(float, 4);
    else DLA_GATE(float, 1);
  }
#undef DLA_GATE
}

void launch_relu2(bool bf16, const void* u, void* y, int64_t n, hipStream_t st) {
  if (n == 0) return;
  const bool vec = n % 8 == 0 && reinterpret_cast<uintptr_t>(u) % 16 == 0 && reinterpret_cast<uintptr_t>(y) % 16 == 0;
  if (bf16) {
    const bf16_t* up = static_cast<const bf16_t*>(u);
    bf16_t* yp = static_cast<bf16_t*>(y);
    if (vec) relu2_kernel<bf16_t, 8><<<grid_for(n / 8), 256, 0, st>>>(up, yp, n);
    else relu2_kernel<bf16_t, 1><<<grid_for(n), 256, 0, st>>>(up, yp, n);
  } else {
    const float* up = static_cast<const float*>(u);
    float* yp = static_cast<float*>(y);
    if (vec) relu2_kernel<float, 8><<<grid_for(n / 8), 256, 0, st>>>(up, yp, n);
    else relu2_kernel<float, 1><<<grid_for(n), 256, 0, st>>>(up, yp, n);
  }
}

}  // namespace dla
