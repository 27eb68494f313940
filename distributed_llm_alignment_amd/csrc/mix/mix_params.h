// Host/device parameter blocks of the mixer kernels.
#pragma once
#include <cstdint>

namespace dla {

struct RetentionParams {
  const void* qkvg;       // [B, T, H (2 dim + 2 vdim)] rows [q | k | v | g], row stride ld, contiguous in T
  int64_t ld;
  void* y;                // [B, T, H vdim]
  float* state;           // [B, H, vdim, dim]
  float* work;            // chunked form: [B, H, nc, vdim, dim]
  const float* decay;     // [2, H]: decay, log2 decay
  const float* cos_t;     // [positions, rot / 2]
  const float* sin_t;
  const int64_t* slot;    // column of the first token on the device (nullptr: base)
  const int* kv_start;    // [B] first real column, or nullptr
  int64_t base;           // column of the first token
  int B, T, H, dim, vdim, rot;
  float eps, kscale;
  int chunk, nc;
  float* osplit;          // decode split: [B, H, vdim] unnormalised outputs
  int* cnt;               // decode split: arrival counters [B, H], zero between launches
  int vsplit;             // decode split: workgroups per (sequence, head)
  int npos;               // rows of the rotary tables
  int fresh;              // the state starts at zero (base == 0)
};

struct LatentParams {
  const void* q;          // [B, T, H (dim + rot)], contiguous
  const void* kv;         // prefill: [B, S, H (dim + vdim)] = [keys | values], contiguous
  const void* kr;         // prefill: rotated key part, [B, S, rot] inside cache rows
  int64_t kr_sb, kr_st;   // its strides
  const void* latent;     // decode: cache [B, Tmax, R + rot]
  int64_t l_sb, l_st;
  const void* kv_up;      // decode: [H (dim + vdim), R]
  void* qcat;             // decode: [B, H, R + rot] query in latent space | rotated part
  void* o;                // [B, T, H vdim]
  float* part_o;          // decode: [B, H, ns, R]
  float* part_ml;         // decode: [B, H, ns, 2]
  const float* cos_t;
  const float* sin_t;
  const int64_t* slot;    // decode: column of the newest token
  const int* kv_start;    // [B] first real column, or nullptr
  int B, T, S, H, dim, rot, vdim, R;
  int q_base, k_base;     // prefill: column of query 0 / key 0
  int window;             // 0: none
  float scale;
  int ns;                 // decode: key splits
  int tcap;               // decode: cache rows
};

struct LruParams {
  const void* yx;         // [B, T, 2 W] rows [y | x] as projected, contiguous
  const void* bias;       // [2 W]
  const void* conv_w;     // [W, taps], last column = the current token
  const void* conv_b;     // [W]
  const void* gates;      // [2 nb, n, n]: the r gate's blocks, then the i gate's; [out, in]
  const void* gates_b;    // [2 nb, n]
  const void* lam;        // [W]
  float* state;           // [B, W]
  void* hist;             // [B, taps, W] ring: column c's x row (no bias) sits at c % taps
  void* out;              // [B, T, W]
  float* cum;             // prefill: [B, T, W] product of decays since the chunk's start
  float* loc;             // prefill: [B, T, W] state with the chunk started at zero
  float* start;           // prefill: [B, nc, W] state at the chunk's start
  const int64_t* slot;    // decode: column of the token
  const int* kv_start;    // [B] first real column, or nullptr
  int64_t base;           // prefill: column of the first token
  float c;                // log a = -c r softplus(lam)
  int B, T, W, taps, nb, n;
  int chunk, nc;
};

struct GlaParams {
  const void* proj;       // [B, T, ld] rows [q | k | v | g | a1 h], contiguous
  int64_t ld;
  const void* a2;         // [H dim, rank]
  const void* a2_b;       // [H dim]
  const void* norm_w;     // [vdim]
  void* y;                // [B, T, H vdim]
  float* state;           // [B, H, vdim, dim]
  float* work;            // chunked form: [B, H, nc, vdim, dim]
  float* cum;             // chunked form: [B, T, H dim] log2 decay since the sub-chunk's start
  float* total;           // chunked form: [B, nc, H dim] log2 decay of a whole chunk
  const int* kv_start;    // [B] first real column, or nullptr
  int64_t base;           // column of the first token
  int B, T, H, dim, vdim, rank;
  float eps, inv_tau, qscale;
  int nc;
  int fresh;              // the state starts at zero (base == 0)
  int vsplit;             // decode: workgroups per (sequence, head)
  float* osplit;          // decode split: [B, H, vdim] unnormalised outputs
  int* cnt;               // decode split: arrival counters [B, H], zero between launches
};

// LDS bytes of the recurrent kernel
inline int64_t gla_recurrent_lds(const GlaParams& p) { return 4ll * (3 * ((p.dim + 3) / 4 * 4) + 2 * p.vdim); }

struct ChunkAttnParams {
  const void* row;        // prepare: projected rows [B, T, ld], contiguous
  int64_t ld;
  const void* bias;       // [ld]
  const void* q_w;        // [H dim]
  const void* k_w;        // [G dim]
  float eps;
  int rot, v_off;         // v_off: column of the values in a projected row
  const float* cos_t;
  const float* sin_t;
  int npos;               // rows of the rotary tables
  void* q;                // [B, T, H, dim]
  void* k;                // prefill: [B, T, G, dim]
  void* v;                // prefill: [B, T, G, vdim]
  void* kc;               // cache [B, G, rows, dim]
  void* vc;               // cache [B, G, rows, vdim]
  void* o;                // [B, T, H vdim]
  float* part_o;          // decode: [B, H, ns, vdim]
  float* part_ml;         // decode: [B, H, ns, 2]
  const int64_t* slot;    // decode: column of the token
  const int* kv_start;    // [B] first real column, or nullptr
  int64_t base;           // prefill: column of the first token
  int B, T, H, G, dim, vdim, rows;
  int chunk;              // > 0; no chunks: a size no sequence reaches
  float scale;
  int ns;                 // decode: key splits
};

struct StreamGemmParams {
  const uint16_t* a;       // [M, K] bf16 contiguous
  const uint16_t* w;       // [N, K] bf16 contiguous
  uint16_t* y;             // [M, N]
  int M, N, K;
  const float* ssq_in;     // [M, nssq] partial sums of squares of a's rows before the norm weight, or nullptr
  int nssq;
  float eps;
  float* x;                // stream epilogue: fp32 [M, N], updated in place
  const uint16_t* norm_w;  // stream epilogue: the next norm's weight, or nullptr
  float offset;
  float* ssq;              // stream epilogue: [M, ceil(N / 16)]
  float alpha;             // post epilogue: x <- alpha x_prev + . + bias
  const float* res_ssq;    // post epilogue: x holds a sum before its norm; [M, nres] partial sums of squares, or nullptr
  int nres;
  const uint16_t* res_w;   // post epilogue: [N] weight of that norm
  const uint16_t* bias;    // post epilogue: [N], or nullptr
  float* yf;               // cap epilogue: fp32 [M, N]
  float cap;
  const int64_t* ids;      // gate epilogue: [M]
  const uint16_t* table;
  int64_t ldt, off, vocab;
};

}  // namespace dla
