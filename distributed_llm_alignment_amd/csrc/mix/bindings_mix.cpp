// torch.ops.dla ops of the mixer library (_C_mix.so): the fp32 residual stream, latent attention and
// retention of per-layer designs. Host-side validation only; bf16 and fp32 tensors.
#include <ATen/ATen.h>
#include <torch/library.h>

#include <algorithm>
#include <cmath>
#include <tuple>

#include "../bind_util.h"
#include "mix_params.h"

namespace dla {

void launch_embed_stream(bool, const int64_t*, const void*, float, float*, int*, int64_t, int64_t, int, hipStream_t);
void launch_stream_norm(bool, float*, const void*, const void*, const float*, const void*, void*, float, float,
                        int64_t, int, hipStream_t);
void launch_side_gate(bool, const void*, const int64_t*, const void*, int64_t, int64_t, void*, int64_t, int, int64_t,
                      hipStream_t);
void launch_relu2(bool, const void*, void*, int64_t, hipStream_t);
int retention_chunk(bool, const RetentionParams&);
void launch_retention_prefill(bool, const RetentionParams&, hipStream_t);
void launch_retention_recurrent(bool, const RetentionParams&, hipStream_t);
void launch_latent_prepare(bool, const void*, int64_t, const void*, const void*, float, void*, void*, int64_t, int64_t,
                           const int64_t*, const int*, const float*, const float*, int, int, int, int, int, int,
                           hipStream_t);
int latent_prefill_waves(bool, const LatentParams&);
bool latent_prefill_mfma_ok(const LatentParams&);
void launch_latent_prefill_mfma(const LatentParams&, hipStream_t);
void launch_latent_prefill_any(bool, const LatentParams&, hipStream_t);
int latent_decode_tile(bool, const LatentParams&);
void launch_latent_decode(bool, const LatentParams&, int, hipStream_t);

void launch_stream_gemm(const StreamGemmParams&, int, hipStream_t);

namespace {

using OptT = c10::optional<at::Tensor>;

// bf16 or fp32 GPU tensor; returns whether it is bf16
bool elem(const at::Tensor& t, const char* name) {
  check_cuda(t, name);
  TORCH_CHECK(t.scalar_type() == at::kBFloat16 || t.scalar_type() == at::kFloat, name, " must be bfloat16 or float32");
  return t.scalar_type() == at::kBFloat16;
}
void like(const at::Tensor& t, const at::Tensor& ref, const char* name) {
  check_cuda(t, name);
  TORCH_CHECK(t.scalar_type() == ref.scalar_type() && t.device() == ref.device(), name, ": dtype / device mismatch");
}
void vec_like(const at::Tensor& t, const at::Tensor& ref, int64_t n, const char* name) {
  like(t, ref, name);
  TORCH_CHECK(t.dim() == 1 && t.size(0) == n && t.is_contiguous(), name, " must be contiguous [", n, "]");
}
void ids_ok(const at::Tensor& ids, const at::Tensor& ref, int64_t n) {
  check_cuda(ids, "ids");
  TORCH_CHECK(ids.scalar_type() == at::kLong && ids.is_contiguous() && ids.numel() == n && ids.device() == ref.device(),
              "ids: contiguous int64, one per row");
}
const int* starts(const OptT& t, const at::Tensor& ref, int64_t B) {
  if (!t.has_value()) return nullptr;
  check_i32(*t, "kv_start");
  TORCH_CHECK(t->dim() == 1 && t->size(0) == B && t->is_contiguous() && t->device() == ref.device(), "kv_start int32 [B]");
  return t->data_ptr<int>();
}
const int64_t* slot_ptr(const at::Tensor& t, const at::Tensor& ref) {
  check_cuda(t, "slot");
  TORCH_CHECK(t.scalar_type() == at::kLong && t.numel() == 1 && t.device() == ref.device(), "slot int64 [1]");
  return t.data_ptr<int64_t>();
}
// cos / sin fp32 [positions, rot / 2]; returns the number of positions
int64_t tables(const at::Tensor& c, const at::Tensor& s, int64_t rot, const at::Tensor& ref) {
  check_f32(c, "cos");
  check_f32(s, "sin");
  TORCH_CHECK(rot >= 0 && rot % 2 == 0, "rot must be even");
  TORCH_CHECK(c.dim() == 2 && c.sizes() == s.sizes() && c.size(1) == rot / 2 && c.is_contiguous() && s.is_contiguous() &&
                  c.device() == ref.device() && s.device() == ref.device(),
              "cos / sin [positions, rot / 2]");
  return c.size(0);
}

at::Tensor embed_stream(const at::Tensor& ids, const at::Tensor& table, double scale, at::Tensor bad) {
  const bool bf = elem(table, "table");
  TORCH_CHECK(table.dim() == 2 && table.is_contiguous(), "table [V, H] contiguous");
  ids_ok(ids, table, ids.numel());
  check_i32(bad, "bad");
  same_device(bad, table);
  c10::hip::HIPGuardMasqueradingAsCUDA guard(table.device());
  auto shape = ids.sizes().vec();
  shape.push_back(table.size(1));
  auto x = at::empty(shape, table.options().dtype(at::kFloat));
  launch_embed_stream(bf, ids.data_ptr<int64_t>(), table.data_ptr(), static_cast<float>(scale), x.data_ptr<float>(),
                      bad.data_ptr<int>(), ids.numel(), table.size(0), static_cast<int>(table.size(1)), cur_stream(table));
  return x;
}

at::Tensor stream_norm(at::Tensor x, const OptT& delta, const OptT& delta_w, const OptT& inject, const OptT& w, double eps,
                       double offset, bool bf16) {
  check_f32(x, "x");
  TORCH_CHECK(x.dim() >= 1 && x.is_contiguous() && x.size(-1) > 0, "x contiguous [.., H]");
  const int64_t H = x.size(-1), rows = x.numel() / H;
  TORCH_CHECK(rows < (1ll << 31) && H < (1 << 24), "x too large");
  auto y = at::empty(x.sizes(), x.options().dtype(bf16 ? at::kBFloat16 : at::kFloat));
  at::Tensor d;
  if (delta.has_value()) {
    d = delta->contiguous();
    like(d, y, "delta");
    TORCH_CHECK(d.numel() == x.numel() && d.size(-1) == H, "delta like x");
  }
  TORCH_CHECK(!delta_w.has_value() || d.defined(), "delta_w without delta");
  if (delta_w.has_value()) vec_like(*delta_w, y, H, "delta_w");
  if (w.has_value()) vec_like(*w, y, H, "w");
  if (inject.has_value()) {
    check_f32(*inject, "inject");
    TORCH_CHECK(inject->sizes() == x.sizes() && inject->is_contiguous() && inject->device() == x.device(), "inject like x");
  }
  check_aligned16(x, "x");
  c10::hip::HIPGuardMasqueradingAsCUDA guard(x.device());
  launch_stream_norm(bf16, x.data_ptr<float>(), d.defined() ? d.data_ptr() : nullptr,
                     delta_w.has_value() ? delta_w->data_ptr() : nullptr,
                     inject.has_value() ? inject->data_ptr<float>() : nullptr, w.has_value() ? w->data_ptr() : nullptr,
                     y.data_ptr(), static_cast<float>(eps), static_cast<float>(offset), rows, static_cast<int>(H), cur_stream(x));
  return y;
}

at::Tensor side_gate(const at::Tensor& z, const at::Tensor& ids, const at::Tensor& table, int64_t off) {
  const bool bf = elem(z, "z");
  like(table, z, "table");
  const int64_t dim = z.size(-1), rows = z.numel() / dim;
  TORCH_CHECK(z.is_contiguous() && table.dim() == 2 && table.stride(1) == 1 && off >= 0 && off + dim <= table.size(1),
              "side_gate: z [.., dim], table [V, >= off + dim]");
  ids_ok(ids, z, rows);
  c10::hip::HIPGuardMasqueradingAsCUDA guard(z.device());
  auto out = at::empty_like(z);
  launch_side_gate(bf, z.data_ptr(), ids.data_ptr<int64_t>(), table.data_ptr(), table.stride(0), off, out.data_ptr(), rows,
                   static_cast<int>(dim), table.size(0), cur_stream(z));
  return out;
}

at::Tensor relu2(const at::Tensor& u_) {
  const bool bf = elem(u_, "u");
  const at::Tensor u = u_.contiguous();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(u.device());
  auto y = at::empty_like(u);
  launch_relu2(bf, u.data_ptr(), y.data_ptr(), u.numel(), cur_stream(u));
  return y;
}

// Decode projection, <= 32 rows (stream_gemm.hip): epi 0 store, 1 relu^2, 2 gate, 3 stream.
std::tuple<at::Tensor, at::Tensor> stream_gemm(const at::Tensor& a, const at::Tensor& w, int64_t epi, const OptT& ssq_in,
                                               double eps, OptT x, const OptT& norm_w, double offset, const OptT& ids,
                                               const OptT& table, int64_t off) {
  check_bf16(a, "a");
  check_bf16(w, "w");
  same_device(a, w);
  TORCH_CHECK(a.dim() == 2 && a.is_contiguous() && w.dim() == 2 && w.is_contiguous() && a.size(1) == w.size(1), "a [M, K], w [N, K]");
  const int64_t M = a.size(0), N = w.size(0), K = w.size(1);
  TORCH_CHECK(M >= 1 && M <= 32 && N >= 1 && N < (1 << 24) && K >= 8 && K < (1 << 24) && K % 8 == 0 && epi >= 0 && epi <= 3,
              "stream_gemm: 1 <= M <= 32, K % 8 == 0");
  check_aligned16(a, "a");
  check_aligned16(w, "w");
  StreamGemmParams p{};
  p.a = cbp(a);
  p.w = cbp(w);
  p.M = static_cast<int>(M);
  p.N = static_cast<int>(N);
  p.K = static_cast<int>(K);
  p.eps = static_cast<float>(eps);
  p.offset = static_cast<float>(offset);
  if (ssq_in.has_value()) {
    check_f32(*ssq_in, "ssq_in");
    TORCH_CHECK(ssq_in->dim() == 2 && ssq_in->size(0) == M && ssq_in->is_contiguous() && ssq_in->device() == a.device(), "ssq_in [M, blocks]");
    p.ssq_in = ssq_in->data_ptr<float>();
    p.nssq = static_cast<int>(ssq_in->size(1));
  }
  c10::hip::HIPGuardMasqueradingAsCUDA guard(a.device());
  auto y = at::empty({M, N}, a.options());
  p.y = bp(y);
  at::Tensor ssq;
  if (epi == 3) {
    TORCH_CHECK(x.has_value(), "stream epilogue: x");
    check_f32(*x, "x");
    TORCH_CHECK(x->numel() == M * N && x->size(-1) == N && x->is_contiguous() && x->device() == a.device(), "x [M, N]");
    p.x = x->data_ptr<float>();
    if (norm_w.has_value()) {
      vec_like(*norm_w, a, N, "norm_w");
      p.norm_w = cbp(*norm_w);
    }
    ssq = at::empty({M, (N + 15) / 16}, x->options());
    p.ssq = ssq.data_ptr<float>();
  } else {
    ssq = at::empty({0}, a.options().dtype(at::kFloat));
  }
  if (epi == 2) {
    TORCH_CHECK(ids.has_value() && table.has_value(), "gate epilogue: ids, table");
    ids_ok(*ids, a, M);
    like(*table, a, "table");
    TORCH_CHECK(table->dim() == 2 && table->stride(1) == 1 && off >= 0 && off + N <= table->size(1), "table [V, >= off + N]");
    p.ids = ids->data_ptr<int64_t>();
    p.table = cbp(*table);
    p.ldt = table->stride(0);
    p.off = off;
    p.vocab = table->size(0);
  }
  launch_stream_gemm(p, static_cast<int>(epi), cur_stream(a));
  return {y, ssq};
}

// ---- retention ----
RetentionParams retention_params(const at::Tensor& qkvg, int64_t H, int64_t dim, int64_t vdim, int64_t rot, double eps,
                                 const at::Tensor& decay, const at::Tensor& state, const OptT& kv_start,
                                 const at::Tensor& cos_t, const at::Tensor& sin_t) {
  elem(qkvg, "qkvg");
  TORCH_CHECK(qkvg.dim() == 3 && qkvg.is_contiguous() && H > 0 && dim > 0 && vdim > 0 &&
                  qkvg.size(2) == 2 * H * (dim + vdim) && rot <= dim,
              "qkvg [B, T, 2 H (dim + vdim)] contiguous");
  const int64_t B = qkvg.size(0), T = qkvg.size(1);
  TORCH_CHECK(B > 0 && T > 0 && B < 65536 && H < 65536 && T < (1ll << 30), "retention: shape");
  check_f32(state, "state");
  check_f32(decay, "decay");
  same_device(qkvg, state);
  same_device(qkvg, decay);
  TORCH_CHECK(state.is_contiguous() && state.sizes() == at::IntArrayRef({B, H, vdim, dim}), "state fp32 [B, H, vdim, dim]");
  TORCH_CHECK(decay.is_contiguous() && decay.sizes() == at::IntArrayRef({2, H}), "decay fp32 [2, H]");
  check_aligned16(state, "state");
  RetentionParams p{};
  p.npos = static_cast<int>(tables(cos_t, sin_t, rot, qkvg));
  p.qkvg = qkvg.data_ptr();
  p.ld = qkvg.size(2);
  p.state = state.data_ptr<float>();
  p.decay = decay.data_ptr<float>();
  p.cos_t = cos_t.data_ptr<float>();
  p.sin_t = sin_t.data_ptr<float>();
  p.kv_start = starts(kv_start, qkvg, B);
  p.B = static_cast<int>(B);
  p.T = static_cast<int>(T);
  p.H = static_cast<int>(H);
  p.dim = static_cast<int>(dim);
  p.vdim = static_cast<int>(vdim);
  p.rot = static_cast<int>(rot);
  p.eps = static_cast<float>(eps);
  p.vsplit = 1;
  p.kscale = 1.f / std::sqrt(static_cast<float>(dim));
  return p;
}

at::Tensor retention_prefill(const at::Tensor& qkvg, int64_t H, int64_t dim, int64_t vdim, int64_t rot, double eps,
                             const at::Tensor& decay, at::Tensor state, const OptT& kv_start, const at::Tensor& cos_t,
                             const at::Tensor& sin_t, int64_t base) {
  RetentionParams p = retention_params(qkvg, H, dim, vdim, rot, eps, decay, state, kv_start, cos_t, sin_t);
  const bool bf = qkvg.scalar_type() == at::kBFloat16;
  TORCH_CHECK(base >= 0 && (rot == 0 || base + p.T <= cos_t.size(0)), "positions exceed the rotary table");
  c10::hip::HIPGuardMasqueradingAsCUDA guard(qkvg.device());
  auto y = at::empty({p.B, p.T, H * vdim}, qkvg.options());
  p.base = base;
  p.fresh = base == 0;
  p.y = y.data_ptr();
  p.chunk = retention_chunk(bf, p);
  if (p.chunk == 0) {
    TORCH_CHECK(2 * (dim + vdim) * 4 + 64 <= 60 * 1024, "retention: head sizes too large");
    launch_retention_recurrent(bf, p, cur_stream(qkvg));
    return y;
  }
  p.nc = (p.T + p.chunk - 1) / p.chunk;
  auto work = at::empty({p.B, H, p.nc, vdim, dim}, state.options());
  p.work = work.data_ptr<float>();
  launch_retention_prefill(bf, p, cur_stream(qkvg));
  return y;
}

at::Tensor retention_decode(const at::Tensor& qkvg, int64_t H, int64_t dim, int64_t vdim, int64_t rot, double eps,
                            const at::Tensor& decay, at::Tensor state, const at::Tensor& slot, const OptT& kv_start,
                            const at::Tensor& cos_t, const at::Tensor& sin_t, const OptT& cnt) {
  RetentionParams p = retention_params(qkvg, H, dim, vdim, rot, eps, decay, state, kv_start, cos_t, sin_t);
  TORCH_CHECK(p.T == 1, "retention_decode: one token per row");
  TORCH_CHECK(2 * (dim + vdim) * 4 + 64 <= 60 * 1024, "retention: head sizes too large");
  c10::hip::HIPGuardMasqueradingAsCUDA guard(qkvg.device());
  auto y = at::empty({p.B, 1, H * vdim}, qkvg.options());
  p.y = y.data_ptr();
  p.slot = slot_ptr(slot, qkvg);
  // few (sequence, head) pairs with a large state (>= 128 KB): several workgroups share the value rows
  // of one pair, >= 32 rows each (smaller states lose more to the hand-off than they gain)
  at::Tensor part;
  if (cnt.has_value() && dim * vdim >= 32 * 1024) {
    check_i32(*cnt, "cnt");
    TORCH_CHECK(cnt->is_contiguous() && cnt->numel() >= p.B * H && cnt->device() == qkvg.device(), "cnt int32, >= B H");
    int64_t vs = std::min<int64_t>(512 / std::max<int64_t>(1, p.B * H), vdim / 32);
    vs = std::min<int64_t>(vs, 8);
    if (vs > 1) {
      part = at::empty({p.B, H, vdim}, state.options());
      p.osplit = part.data_ptr<float>();
      p.cnt = cnt->data_ptr<int>();
      p.vsplit = static_cast<int>(vs);
    }
  }
  launch_retention_recurrent(qkvg.scalar_type() == at::kBFloat16, p, cur_stream(qkvg));
  return y;
}

// ---- latent attention ----
void cache_ok(const at::Tensor& latent, const at::Tensor& ref, int64_t B, int64_t width) {
  like(latent, ref, "latent");
  TORCH_CHECK(latent.dim() == 3 && latent.size(0) == B && latent.size(2) == width && latent.stride(2) == 1,
              "latent cache [B, T_max, kv_rank + rot]");
}

at::Tensor latent_prepare(const at::Tensor& down, const at::Tensor& qw, const at::Tensor& kw, double eps,
                          at::Tensor latent, const at::Tensor& slot, const OptT& kv_start, const at::Tensor& cos_t,
                          const at::Tensor& sin_t) {
  const bool bf = elem(down, "down");
  const int64_t qr = qw.numel(), R = kw.numel();
  TORCH_CHECK(down.dim() == 3 && down.is_contiguous() && down.size(2) >= qr + R && qr > 0 && R > 0, "down [B, T, qr + R + rot]");
  const int64_t B = down.size(0), T = down.size(1), rot = down.size(2) - qr - R;
  vec_like(qw, down, qr, "q_norm_w");
  vec_like(kw, down, R, "kv_norm_w");
  cache_ok(latent, down, B, R + rot);
  const int64_t n = tables(cos_t, sin_t, rot, down);
  // the column is on the device: the caller's cache bounds it; the tables cover the whole cache
  TORCH_CHECK(T <= latent.size(1) && (rot == 0 || n >= latent.size(1)), "rotary table shorter than the cache");
  TORCH_CHECK(B * T < (1ll << 31), "too many rows");
  c10::hip::HIPGuardMasqueradingAsCUDA guard(down.device());
  auto cq = at::empty({B, T, qr}, down.options());
  launch_latent_prepare(bf, down.data_ptr(), down.size(2), qw.data_ptr(), kw.data_ptr(), static_cast<float>(eps),
                        cq.data_ptr(), latent.data_ptr(), latent.stride(0), latent.stride(1), slot_ptr(slot, down),
                        starts(kv_start, down, B), cos_t.data_ptr<float>(), sin_t.data_ptr<float>(),
                        static_cast<int>(B), static_cast<int>(T), static_cast<int>(qr), static_cast<int>(R),
                        static_cast<int>(rot), static_cast<int>(latent.size(1)), cur_stream(down));
  return cq;
}

LatentParams latent_sizes(int64_t B, int64_t T, int64_t H, int64_t dim, int64_t rot, int64_t vdim, double scale,
                          int64_t window) {
  TORCH_CHECK(B > 0 && T > 0 && H > 0 && dim > 0 && rot >= 0 && vdim > 0 && window >= 0 && B < 65536 && H < 65536 &&
                  T < (1ll << 30) && window < (1ll << 31),
              "latent attention: shape");
  LatentParams p{};
  p.B = static_cast<int>(B);
  p.T = static_cast<int>(T);
  p.H = static_cast<int>(H);
  p.dim = static_cast<int>(dim);
  p.rot = static_cast<int>(rot);
  p.vdim = static_cast<int>(vdim);
  p.scale = static_cast<float>(scale);
  p.window = static_cast<int>(window);
  return p;
}

at::Tensor latent_prefill(const at::Tensor& q, const at::Tensor& kv, const at::Tensor& kr, int64_t H, int64_t dim,
                          int64_t rot, int64_t vdim, double scale, int64_t window, const OptT& kv_start,
                          const at::Tensor& cos_t, const at::Tensor& sin_t, int64_t q_base, int64_t k_base) {
  const bool bf = elem(q, "q");
  TORCH_CHECK(q.dim() == 3 && q.is_contiguous() && q.size(2) == H * (dim + rot), "q [B, T, H (dim + rot)] contiguous");
  LatentParams p = latent_sizes(q.size(0), q.size(1), H, dim, rot, vdim, scale, window);
  like(kv, q, "kv");
  like(kr, q, "kr");
  TORCH_CHECK(kv.dim() == 3 && kv.is_contiguous() && kv.size(0) == p.B && kv.size(2) == H * (dim + vdim),
              "kv [B, S, H (dim + vdim)] contiguous");
  TORCH_CHECK(kr.dim() == 3 && kr.size(0) == p.B && kr.size(1) == kv.size(1) && kr.size(2) == rot &&
                  (rot == 0 || kr.stride(2) == 1),
              "kr [B, S, rot]");
  TORCH_CHECK(kv.size(1) > 0 && kv.size(1) < (1ll << 30) && q_base >= 0 && k_base >= 0 && q_base + p.T < (1ll << 30),
              "latent_prefill: columns");
  const int64_t n = tables(cos_t, sin_t, rot, q);
  TORCH_CHECK(rot == 0 || q_base + p.T <= n, "positions exceed the rotary table");
  p.q = q.data_ptr();
  p.kv = kv.data_ptr();
  p.kr = kr.data_ptr();
  p.kr_sb = kr.stride(0);
  p.kr_st = kr.stride(1);
  p.S = static_cast<int>(kv.size(1));
  p.q_base = static_cast<int>(q_base);
  p.k_base = static_cast<int>(k_base);
  p.kv_start = starts(kv_start, q, p.B);
  p.cos_t = cos_t.data_ptr<float>();
  p.sin_t = sin_t.data_ptr<float>();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(q.device());
  auto o = at::empty({p.B, p.T, H * vdim}, q.options());
  p.o = o.data_ptr();
  if (bf && latent_prefill_mfma_ok(p)) {
    launch_latent_prefill_mfma(p, cur_stream(q));
    return o;
  }
  TORCH_CHECK(latent_prefill_waves(bf, p) > 0, "latent attention: head sizes too large");
  launch_latent_prefill_any(bf, p, cur_stream(q));
  return o;
}

at::Tensor latent_decode(const at::Tensor& q, const at::Tensor& latent, const at::Tensor& kv_up, int64_t H, int64_t dim,
                         int64_t rot, int64_t vdim, double scale, int64_t window, const at::Tensor& slot,
                         const OptT& kv_start, const at::Tensor& cos_t, const at::Tensor& sin_t) {
  const bool bf = elem(q, "q");
  TORCH_CHECK(q.dim() == 3 && q.size(1) == 1 && q.is_contiguous() && q.size(2) == H * (dim + rot),
              "q [B, 1, H (dim + rot)] contiguous");
  LatentParams p = latent_sizes(q.size(0), 1, H, dim, rot, vdim, scale, window);
  like(kv_up, q, "kv_up");
  TORCH_CHECK(kv_up.dim() == 2 && kv_up.is_contiguous() && kv_up.size(0) == H * (dim + vdim), "kv_up [H (dim + vdim), R]");
  p.R = static_cast<int>(kv_up.size(1));
  cache_ok(latent, q, p.B, p.R + rot);
  const int64_t n = tables(cos_t, sin_t, rot, q);
  TORCH_CHECK(rot == 0 || n >= latent.size(1), "rotary table shorter than the cache");
  p.q = q.data_ptr();
  p.latent = latent.data_ptr();
  p.l_sb = latent.stride(0);
  p.l_st = latent.stride(1);
  p.tcap = static_cast<int>(latent.size(1));
  p.kv_up = kv_up.data_ptr();
  p.slot = slot_ptr(slot, q);
  p.kv_start = starts(kv_start, q, p.B);
  p.cos_t = cos_t.data_ptr<float>();
  p.sin_t = sin_t.data_ptr<float>();
  const int tile = latent_decode_tile(bf, p);
  TORCH_CHECK(tile > 0 && 4 * p.R <= 48 * 1024, "latent attention: latent too wide");
  // enough key splits to fill the chip, none shorter than a tile of the longest visible range
  int64_t most = latent.size(1);
  if (window > 0 && window < most) most = window;
  const int64_t groups = static_cast<int64_t>(p.B) * ((H + 15) / 16);
  int64_t ns = (512 + groups - 1) / groups;
  ns = std::min<int64_t>(ns, (most + tile - 1) / tile);
  p.ns = static_cast<int>(std::max<int64_t>(1, std::min<int64_t>(ns, 256)));
  c10::hip::HIPGuardMasqueradingAsCUDA guard(q.device());
  auto qcat = at::empty({p.B, H, p.R + rot}, q.options());
  auto po = at::empty({p.B, H, p.ns, p.R}, q.options().dtype(at::kFloat));
  auto ml = at::empty({p.B, H, p.ns, 2}, po.options());
  auto o = at::empty({p.B, 1, H * vdim}, q.options());
  p.qcat = qcat.data_ptr();
  p.part_o = po.data_ptr<float>();
  p.part_ml = ml.data_ptr<float>();
  p.o = o.data_ptr();
  launch_latent_decode(bf, p, tile, cur_stream(q));
  return o;
}

}  // namespace
}  // namespace dla

TORCH_LIBRARY_FRAGMENT(dla, m) {
  m.def("embed_stream(Tensor ids, Tensor table, float scale, Tensor(a!) bad) -> Tensor");
  m.def("stream_norm(Tensor(a!) x, Tensor? delta, Tensor? delta_w, Tensor? inject, Tensor? w, float eps, float offset, bool bf16) -> Tensor");
  m.def("side_gate(Tensor z, Tensor ids, Tensor table, int off) -> Tensor");
  m.def("stream_gemm(Tensor a, Tensor w, int epi, Tensor? ssq_in, float eps, Tensor(a!)? x, Tensor? norm_w, float offset, Tensor? ids, Tensor? table, int off) -> (Tensor, Tensor)");
  m.def("relu2(Tensor u) -> Tensor");
  m.def("retention_prefill(Tensor qkvg, int H, int dim, int vdim, int rot, float eps, Tensor decay, Tensor(a!) state, Tensor? kv_start, Tensor cos, Tensor sin, int base) -> Tensor");
  m.def("retention_decode(Tensor qkvg, int H, int dim, int vdim, int rot, float eps, Tensor decay, Tensor(a!) state, Tensor slot, Tensor? kv_start, Tensor cos, Tensor sin, Tensor(b!)? cnt) -> Tensor");
  m.def("latent_prepare(Tensor down, Tensor q_norm_w, Tensor kv_norm_w, float eps, Tensor(a!) latent, Tensor slot, Tensor? kv_start, Tensor cos, Tensor sin) -> Tensor");
  m.def("latent_prefill(Tensor q, Tensor kv, Tensor kr, int H, int dim, int rot, int vdim, float scale, int window, Tensor? kv_start, Tensor cos, Tensor sin, int q_base, int k_base) -> Tensor");
  m.def("latent_decode(Tensor q, Tensor latent, Tensor kv_up, int H, int dim, int rot, int vdim, float scale, int window, Tensor slot, Tensor? kv_start, Tensor cos, Tensor sin) -> Tensor");
}

TORCH_LIBRARY_IMPL(dla, CUDA, m) {
  m.impl("embed_stream", &dla::embed_stream);
  m.impl("stream_norm", &dla::stream_norm);
  m.impl("side_gate", &dla::side_gate);
  m.impl("stream_gemm", &dla::stream_gemm);
  m.impl("relu2", &dla::relu2);
  m.impl("retention_prefill", &dla::retention_prefill);
  m.impl("retention_decode", &dla::retention_decode);
  m.impl("latent_prepare", &dla::latent_prepare);
  m.impl("latent_prefill", &dla::latent_prefill);
  m.impl("latent_decode", &dla::latent_decode);
}
