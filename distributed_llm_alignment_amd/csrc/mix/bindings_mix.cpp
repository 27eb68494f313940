// torch.ops.dla ops of the mixer library (_C_mix.so): the fp32 residual stream and the mixers of
// per-layer designs. Host-side validation only; bf16 and fp32 tensors.
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

void launch_post_norm(bool, float*, const void*, const void*, float, const void*, const void*, void*, float, int64_t, int,
                      hipStream_t);
void launch_geglu(bool, const void*, void*, int64_t, int, hipStream_t);
void launch_softcap(bool, const void*, float*, int64_t, float, hipStream_t);
int lru_chunk(const LruParams&);
void launch_lru_prefill(bool, const LruParams&, hipStream_t);
void launch_lru_decode(bool, const LruParams&, hipStream_t);
int gla_chunks(bool, const GlaParams&);
void launch_gla_prefill(const GlaParams&, hipStream_t);
void launch_gla_recurrent(bool, const GlaParams&, hipStream_t);
void launch_chunk_prepare(bool, const ChunkAttnParams&, bool, hipStream_t);
void launch_chunk_store(bool, const ChunkAttnParams&, hipStream_t);
bool chunk_prefill_mfma_ok(const ChunkAttnParams&);
void launch_chunk_prefill_mfma(const ChunkAttnParams&, hipStream_t);
void launch_chunk_prefill_any(bool, const ChunkAttnParams&, hipStream_t);
void launch_chunk_decode(bool, const ChunkAttnParams&, hipStream_t);

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

at::Tensor post_norm(at::Tensor x, const OptT& delta, const OptT& bias, double alpha, const at::Tensor& w, const OptT& w2,
                     double eps, bool bf16) {
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
  vec_like(w, y, H, "w");
  if (bias.has_value()) vec_like(*bias, y, H, "bias");
  if (w2.has_value()) vec_like(*w2, y, H, "w2");
  check_aligned16(x, "x");
  c10::hip::HIPGuardMasqueradingAsCUDA guard(x.device());
  launch_post_norm(bf16, x.data_ptr<float>(), d.defined() ? d.data_ptr() : nullptr, bias.has_value() ? bias->data_ptr() : nullptr,
                   static_cast<float>(alpha), w.data_ptr(), w2.has_value() ? w2->data_ptr() : nullptr, y.data_ptr(),
                   static_cast<float>(eps), rows, static_cast<int>(H), cur_stream(x));
  return y;
}

at::Tensor geglu(const at::Tensor& u_) {
  const bool bf = elem(u_, "u");
  const at::Tensor u = u_.contiguous();
  TORCH_CHECK(u.dim() >= 1 && u.size(-1) > 0 && u.size(-1) % 2 == 0 && u.size(-1) < (1ll << 31), "geglu: u [.., 2 F]");
  c10::hip::HIPGuardMasqueradingAsCUDA guard(u.device());
  auto shape = u.sizes().vec();
  shape.back() /= 2;
  auto y = at::empty(shape, u.options());
  launch_geglu(bf, u.data_ptr(), y.data_ptr(), y.numel() / shape.back(), static_cast<int>(shape.back()), cur_stream(u));
  return y;
}

at::Tensor softcap(const at::Tensor& z_, double cap) {
  const bool bf = elem(z_, "z");
  TORCH_CHECK(cap > 0, "softcap: cap > 0");
  const at::Tensor z = z_.contiguous();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(z.device());
  auto y = at::empty(z.sizes(), z.options().dtype(at::kFloat));
  launch_softcap(bf, z.data_ptr(), y.data_ptr<float>(), z.numel(), static_cast<float>(cap), cur_stream(z));
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

// Decode projections, <= 32 rows (stream_gemm.hip)
StreamGemmParams gemm_params(const at::Tensor& a, const at::Tensor& w, int64_t per_col, const OptT& ssq_in, double eps) {
  check_bf16(a, "a");
  check_bf16(w, "w");
  same_device(a, w);
  TORCH_CHECK(a.dim() == 2 && a.is_contiguous() && w.dim() == 2 && w.is_contiguous() && a.size(1) == w.size(1), "a [M, K], w [N, K]");
  const int64_t M = a.size(0), N = w.size(0) / per_col, K = w.size(1);
  TORCH_CHECK(M >= 1 && M <= 32 && N >= 1 && N < (1 << 24) && w.size(0) == N * per_col && K >= 8 && K < (1 << 24) && K % 8 == 0,
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
  if (ssq_in.has_value()) {
    check_f32(*ssq_in, "ssq_in");
    TORCH_CHECK(ssq_in->dim() == 2 && ssq_in->size(0) == M && ssq_in->is_contiguous() && ssq_in->device() == a.device(), "ssq_in [M, blocks]");
    p.ssq_in = ssq_in->data_ptr<float>();
    p.nssq = static_cast<int>(ssq_in->size(1));
  }
  return p;
}

// the fp32 stream and the partial sums of squares of an epilogue that updates it; returns ssq
at::Tensor gemm_stream(StreamGemmParams& p, const at::Tensor& a, const at::Tensor& x, const OptT& norm_w) {
  check_f32(x, "x");
  TORCH_CHECK(x.numel() == static_cast<int64_t>(p.M) * p.N && x.size(-1) == p.N && x.is_contiguous() && x.device() == a.device(), "x [M, N]");
  p.x = x.data_ptr<float>();
  if (norm_w.has_value()) {
    vec_like(*norm_w, a, p.N, "norm_w");
    p.norm_w = cbp(*norm_w);
  }
  auto ssq = at::empty({p.M, (p.N + 15) / 16}, x.options());
  p.ssq = ssq.data_ptr<float>();
  return ssq;
}

// epi 0 store, 1 relu^2, 2 gate, 3 stream, 5 gelu-gated unit (w = [gate; up])
std::tuple<at::Tensor, at::Tensor> stream_gemm(const at::Tensor& a, const at::Tensor& w, int64_t epi, const OptT& ssq_in,
                                               double eps, OptT x, const OptT& norm_w, double offset, const OptT& ids,
                                               const OptT& table, int64_t off) {
  TORCH_CHECK((epi >= 0 && epi <= 3) || epi == 5, "stream_gemm: epilogue");
  StreamGemmParams p = gemm_params(a, w, epi == 5 ? 2 : 1, ssq_in, eps);
  p.offset = static_cast<float>(offset);
  c10::hip::HIPGuardMasqueradingAsCUDA guard(a.device());
  auto y = at::empty({p.M, p.N}, a.options());
  p.y = bp(y);
  at::Tensor ssq;
  if (epi == 3) {
    TORCH_CHECK(x.has_value(), "stream epilogue: x");
    ssq = gemm_stream(p, a, *x, norm_w);
  } else {
    ssq = at::empty({0}, a.options().dtype(at::kFloat));
  }
  if (epi == 2) {
    TORCH_CHECK(ids.has_value() && table.has_value(), "gate epilogue: ids, table");
    ids_ok(*ids, a, p.M);
    like(*table, a, "table");
    TORCH_CHECK(table->dim() == 2 && table->stride(1) == 1 && off >= 0 && off + p.N <= table->size(1), "table [V, >= off + N]");
    p.ids = ids->data_ptr<int64_t>();
    p.table = cbp(*table);
    p.ldt = table->stride(0);
    p.off = off;
    p.vocab = table->size(0);
  }
  launch_stream_gemm(p, static_cast<int>(epi), cur_stream(a));
  return {y, ssq};
}

// x <- alpha x_prev + a w^T + bias (x_prev: x normed with res_ssq / res_w, or x itself); returns (bf16(x * norm_w), ssq)
std::tuple<at::Tensor, at::Tensor> stream_gemm_post(const at::Tensor& a, const at::Tensor& w, at::Tensor x, double alpha,
                                                    const OptT& bias, const OptT& res_ssq, const OptT& res_w,
                                                    const at::Tensor& norm_w, double eps) {
  StreamGemmParams p = gemm_params(a, w, 1, c10::nullopt, eps);
  c10::hip::HIPGuardMasqueradingAsCUDA guard(a.device());
  auto y = at::empty({p.M, p.N}, a.options());
  p.y = bp(y);
  at::Tensor ssq = gemm_stream(p, a, x, norm_w);
  p.alpha = static_cast<float>(alpha);
  if (bias.has_value()) {
    vec_like(*bias, a, p.N, "bias");
    p.bias = cbp(*bias);
  }
  TORCH_CHECK(res_ssq.has_value() == res_w.has_value(), "res_ssq and res_w come together");
  if (res_ssq.has_value()) {
    check_f32(*res_ssq, "res_ssq");
    TORCH_CHECK(res_ssq->dim() == 2 && res_ssq->size(0) == p.M && res_ssq->is_contiguous() && res_ssq->device() == a.device(), "res_ssq [M, blocks]");
    vec_like(*res_w, a, p.N, "res_w");
    p.res_ssq = res_ssq->data_ptr<float>();
    p.nres = static_cast<int>(res_ssq->size(1));
    p.res_w = cbp(*res_w);
  }
  launch_stream_gemm(p, 4, cur_stream(a));
  return {y, ssq};
}

// fp32 cap * tanh(a w^T / cap)
at::Tensor stream_gemm_cap(const at::Tensor& a, const at::Tensor& w, double cap) {
  TORCH_CHECK(cap > 0, "cap > 0");
  StreamGemmParams p = gemm_params(a, w, 1, c10::nullopt, 0.0);
  c10::hip::HIPGuardMasqueradingAsCUDA guard(a.device());
  auto y = at::empty({p.M, p.N}, a.options().dtype(at::kFloat));
  p.yf = y.data_ptr<float>();
  p.cap = static_cast<float>(cap);
  launch_stream_gemm(p, 6, cur_stream(a));
  return y;
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

// ---- gated linear recurrence ----
LruParams lru_params(const at::Tensor& yx, const at::Tensor& bias, const at::Tensor& conv_w, const at::Tensor& conv_b,
                     const at::Tensor& gates, const at::Tensor& gates_b, const at::Tensor& lam, double c,
                     const at::Tensor& state, const at::Tensor& hist, const OptT& kv_start) {
  elem(yx, "yx");
  like(conv_w, yx, "conv_w");
  TORCH_CHECK(conv_w.dim() == 2 && conv_w.is_contiguous() && conv_w.size(0) > 0 && conv_w.size(1) > 0 && conv_w.size(1) < 1024,
              "conv_w [W, taps]");
  const int64_t W = conv_w.size(0), taps = conv_w.size(1);
  TORCH_CHECK(yx.dim() == 3 && yx.is_contiguous() && yx.size(2) == 2 * W, "yx [B, T, 2 W] contiguous");
  const int64_t B = yx.size(0), T = yx.size(1);
  TORCH_CHECK(B > 0 && T > 0 && B < 65536 && T < (1ll << 30) && W < (1ll << 24), "lru: shape");
  vec_like(bias, yx, 2 * W, "bias");
  vec_like(conv_b, yx, W, "conv_b");
  vec_like(lam, yx, W, "lam");
  like(gates, yx, "gates");
  like(gates_b, yx, "gates_b");
  TORCH_CHECK(gates.dim() == 3 && gates.is_contiguous() && gates.size(0) > 0 && gates.size(0) % 2 == 0 &&
                  gates.size(1) == gates.size(2) && gates.size(0) / 2 * gates.size(1) == W,
              "gates [2 blocks, n, n], blocks * n = W");
  TORCH_CHECK(gates_b.is_contiguous() && gates_b.sizes() == at::IntArrayRef({gates.size(0), gates.size(1)}), "gates_b [2 blocks, n]");
  check_f32(state, "state");
  same_device(yx, state);
  TORCH_CHECK(state.is_contiguous() && state.sizes() == at::IntArrayRef({B, W}), "state fp32 [B, W]");
  like(hist, yx, "hist");
  TORCH_CHECK(hist.is_contiguous() && hist.sizes() == at::IntArrayRef({B, taps, W}), "hist [B, taps, W]");
  LruParams p{};
  p.yx = yx.data_ptr();
  p.bias = bias.data_ptr();
  p.conv_w = conv_w.data_ptr();
  p.conv_b = conv_b.data_ptr();
  p.gates = gates.data_ptr();
  p.gates_b = gates_b.data_ptr();
  p.lam = lam.data_ptr();
  p.state = state.data_ptr<float>();
  p.hist = hist.data_ptr();
  p.kv_start = starts(kv_start, yx, B);
  p.c = static_cast<float>(c);
  p.B = static_cast<int>(B);
  p.T = static_cast<int>(T);
  p.W = static_cast<int>(W);
  p.taps = static_cast<int>(taps);
  p.nb = static_cast<int>(gates.size(0) / 2);
  p.n = static_cast<int>(gates.size(1));
  TORCH_CHECK(static_cast<int64_t>(p.nb) * ((p.n + 127) / 128) < 65536, "lru: too many gate blocks");
  return p;
}

at::Tensor lru_prefill(const at::Tensor& yx, const at::Tensor& bias, const at::Tensor& conv_w, const at::Tensor& conv_b,
                       const at::Tensor& gates, const at::Tensor& gates_b, const at::Tensor& lam, double c, at::Tensor state,
                       at::Tensor hist, const OptT& kv_start, int64_t base) {
  LruParams p = lru_params(yx, bias, conv_w, conv_b, gates, gates_b, lam, c, state, hist, kv_start);
  TORCH_CHECK(base >= 0 && base < (1ll << 40) && (p.T + 3) / 4 < 65536, "lru_prefill: portion too long");
  c10::hip::HIPGuardMasqueradingAsCUDA guard(yx.device());
  auto out = at::empty({p.B, p.T, p.W}, yx.options());
  p.out = out.data_ptr();
  p.base = base;
  p.chunk = lru_chunk(p);
  p.nc = (p.T + p.chunk - 1) / p.chunk;
  auto cum = at::empty({p.B, p.T, p.W}, state.options()), loc = at::empty({p.B, p.T, p.W}, state.options());
  auto start = at::empty({p.B, p.nc, p.W}, state.options());
  p.cum = cum.data_ptr<float>();
  p.loc = loc.data_ptr<float>();
  p.start = start.data_ptr<float>();
  launch_lru_prefill(yx.scalar_type() == at::kBFloat16, p, cur_stream(yx));
  return out;
}

at::Tensor lru_decode(const at::Tensor& yx, const at::Tensor& bias, const at::Tensor& conv_w, const at::Tensor& conv_b,
                      const at::Tensor& gates, const at::Tensor& gates_b, const at::Tensor& lam, double c, at::Tensor state,
                      at::Tensor hist, const at::Tensor& slot, const OptT& kv_start) {
  LruParams p = lru_params(yx, bias, conv_w, conv_b, gates, gates_b, lam, c, state, hist, kv_start);
  TORCH_CHECK(p.T == 1, "lru_decode: one token per row");
  c10::hip::HIPGuardMasqueradingAsCUDA guard(yx.device());
  auto out = at::empty({p.B, 1, p.W}, yx.options());
  p.out = out.data_ptr();
  p.slot = slot_ptr(slot, yx);
  launch_lru_decode(yx.scalar_type() == at::kBFloat16, p, cur_stream(yx));
  return out;
}

// ---- gated linear attention ----
GlaParams gla_params(const at::Tensor& proj, const at::Tensor& a2, const at::Tensor& a2_b, const at::Tensor& norm_w, int64_t H,
                     int64_t dim, int64_t vdim, double tau, double eps, const at::Tensor& state) {
  elem(proj, "proj");
  like(a2, proj, "a2");
  TORCH_CHECK(a2.dim() == 2 && a2.is_contiguous() && H > 0 && dim > 0 && vdim > 0 && a2.size(0) == H * dim && a2.size(1) > 0 && tau > 0,
              "a2 [H dim, rank]");
  TORCH_CHECK(proj.dim() == 3 && proj.is_contiguous() && proj.size(2) == 2 * H * (dim + vdim) + a2.size(1),
              "proj [B, T, 2 H (dim + vdim) + rank] contiguous");
  const int64_t B = proj.size(0), T = proj.size(1);
  TORCH_CHECK(B > 0 && T > 0 && B < 65536 && H < 65536 && T < (1ll << 30) && H * dim < (1ll << 21), "gla: shape");
  vec_like(a2_b, proj, H * dim, "a2_b");
  vec_like(norm_w, proj, vdim, "norm_w");
  check_f32(state, "state");
  same_device(proj, state);
  TORCH_CHECK(state.is_contiguous() && state.sizes() == at::IntArrayRef({B, H, vdim, dim}), "state fp32 [B, H, vdim, dim]");
  check_aligned16(state, "state");
  GlaParams p{};
  p.proj = proj.data_ptr();
  p.ld = proj.size(2);
  p.a2 = a2.data_ptr();
  p.a2_b = a2_b.data_ptr();
  p.norm_w = norm_w.data_ptr();
  p.state = state.data_ptr<float>();
  p.B = static_cast<int>(B);
  p.T = static_cast<int>(T);
  p.H = static_cast<int>(H);
  p.dim = static_cast<int>(dim);
  p.vdim = static_cast<int>(vdim);
  p.rank = static_cast<int>(a2.size(1));
  p.eps = static_cast<float>(eps);
  p.inv_tau = static_cast<float>(1.0 / tau);
  p.qscale = 1.f / std::sqrt(static_cast<float>(dim));
  p.vsplit = 1;
  TORCH_CHECK(gla_recurrent_lds(p) <= 60 * 1024, "gla: head sizes too large");
  return p;
}

at::Tensor gla_prefill(const at::Tensor& proj, const at::Tensor& a2, const at::Tensor& a2_b, const at::Tensor& norm_w, int64_t H,
                       int64_t dim, int64_t vdim, double tau, double eps, at::Tensor state, const OptT& kv_start, int64_t base) {
  GlaParams p = gla_params(proj, a2, a2_b, norm_w, H, dim, vdim, tau, eps, state);
  TORCH_CHECK(base >= 0 && base < (1ll << 40), "gla_prefill: base");
  const bool bf = proj.scalar_type() == at::kBFloat16;
  c10::hip::HIPGuardMasqueradingAsCUDA guard(proj.device());
  auto y = at::empty({p.B, p.T, H * vdim}, proj.options());
  p.y = y.data_ptr();
  p.base = base;
  p.fresh = base == 0;
  p.kv_start = starts(kv_start, proj, p.B);
  p.nc = gla_chunks(bf, p);
  if (p.nc == 0) {
    launch_gla_recurrent(bf, p, cur_stream(proj));
    return y;
  }
  auto work = at::empty({p.B, H, p.nc, vdim, dim}, state.options());
  auto cum = at::empty({p.B, p.T, H * dim}, state.options()), total = at::empty({p.B, p.nc, H * dim}, state.options());
  p.work = work.data_ptr<float>();
  p.cum = cum.data_ptr<float>();
  p.total = total.data_ptr<float>();
  launch_gla_prefill(p, cur_stream(proj));
  return y;
}

at::Tensor gla_decode(const at::Tensor& proj, const at::Tensor& a2, const at::Tensor& a2_b, const at::Tensor& norm_w, int64_t H,
                      int64_t dim, int64_t vdim, double tau, double eps, at::Tensor state, const OptT& cnt) {
  GlaParams p = gla_params(proj, a2, a2_b, norm_w, H, dim, vdim, tau, eps, state);
  TORCH_CHECK(p.T == 1, "gla_decode: one token per row");
  c10::hip::HIPGuardMasqueradingAsCUDA guard(proj.device());
  auto y = at::empty({p.B, 1, H * vdim}, proj.options());
  p.y = y.data_ptr();
  // few (sequence, head) pairs with a large state (>= 128 KB): several workgroups share the value rows
  at::Tensor part;
  if (cnt.has_value() && dim * vdim >= 32 * 1024) {
    check_i32(*cnt, "cnt");
    TORCH_CHECK(cnt->is_contiguous() && cnt->numel() >= p.B * H && cnt->device() == proj.device(), "cnt int32, >= B H");
    int64_t vs = std::min<int64_t>(512 / std::max<int64_t>(1, p.B * H), vdim / 32);
    vs = std::min<int64_t>(vs, 8);
    if (vs > 1) {
      part = at::empty({p.B, H, vdim}, state.options());
      p.osplit = part.data_ptr<float>();
      p.cnt = cnt->data_ptr<int>();
      p.vsplit = static_cast<int>(vs);
    }
  }
  launch_gla_recurrent(proj.scalar_type() == at::kBFloat16, p, cur_stream(proj));
  return y;
}

// ---- attention inside chunks ----
constexpr int64_t kNoChunks = 1 << 30;

ChunkAttnParams chunk_sizes(int64_t B, int64_t T, int64_t H, int64_t G, int64_t dim, int64_t vdim, int64_t chunk, double scale) {
  TORCH_CHECK(B > 0 && T > 0 && H > 0 && G > 0 && H % G == 0 && dim > 0 && vdim > 0 && chunk >= 0 && chunk <= kNoChunks && B < 65536 &&
                  H < 65536 && T < (1ll << 30) && B * T < (1ll << 31) && dim + vdim <= 4096,
              "chunk attention: shape");
  ChunkAttnParams p{};
  p.B = static_cast<int>(B);
  p.T = static_cast<int>(T);
  p.H = static_cast<int>(H);
  p.G = static_cast<int>(G);
  p.dim = static_cast<int>(dim);
  p.vdim = static_cast<int>(vdim);
  p.chunk = static_cast<int>(chunk > 0 ? chunk : kNoChunks);
  p.scale = static_cast<float>(scale);
  return p;
}

void chunk_row(ChunkAttnParams& p, const at::Tensor& row, const at::Tensor& bias, const at::Tensor& q_w, const at::Tensor& k_w,
               int64_t rot, int64_t v_off, double eps, const at::Tensor& cos_t, const at::Tensor& sin_t) {
  const int64_t nq = static_cast<int64_t>(p.H) * p.dim, nk = static_cast<int64_t>(p.G) * p.dim, nv = static_cast<int64_t>(p.G) * p.vdim;
  TORCH_CHECK(row.is_contiguous() && row.size(2) >= nq + nk && v_off >= 0 && v_off + nv <= row.size(2) && rot >= 0 && rot <= p.dim,
              "row [B, T, >= (H + G) dim] with the values at v_off");
  vec_like(bias, row, row.size(2), "bias");
  vec_like(q_w, row, nq, "q_w");
  vec_like(k_w, row, nk, "k_w");
  p.row = row.data_ptr();
  p.ld = row.size(2);
  p.bias = bias.data_ptr();
  p.q_w = q_w.data_ptr();
  p.k_w = k_w.data_ptr();
  p.eps = static_cast<float>(eps);
  p.rot = static_cast<int>(rot);
  p.v_off = static_cast<int>(v_off);
  p.npos = static_cast<int>(tables(cos_t, sin_t, rot, row));
  p.cos_t = cos_t.data_ptr<float>();
  p.sin_t = sin_t.data_ptr<float>();
}

void chunk_cache(ChunkAttnParams& p, const at::Tensor& kc, const at::Tensor& vc, const at::Tensor& ref) {
  like(kc, ref, "kc");
  like(vc, ref, "vc");
  TORCH_CHECK(kc.dim() == 4 && kc.is_contiguous() && vc.is_contiguous() && kc.size(2) > 0 && kc.size(2) < (1ll << 30) &&
                  kc.sizes() == at::IntArrayRef({p.B, p.G, kc.size(2), p.dim}) &&
                  vc.sizes() == at::IntArrayRef({p.B, p.G, kc.size(2), p.vdim}),
              "cache [B, G, rows, dim] / [B, G, rows, vdim] contiguous");
  p.rows = static_cast<int>(kc.size(2));
  p.kc = kc.data_ptr();
  p.vc = vc.data_ptr();
}

std::tuple<at::Tensor, at::Tensor, at::Tensor> chunk_prepare(const at::Tensor& row, const at::Tensor& bias, const at::Tensor& q_w,
                                                             const at::Tensor& k_w, int64_t H, int64_t G, int64_t dim,
                                                             int64_t vdim, int64_t rot, int64_t v_off, double eps,
                                                             const OptT& kv_start, const at::Tensor& cos_t,
                                                             const at::Tensor& sin_t, int64_t base) {
  const bool bf = elem(row, "row");
  TORCH_CHECK(row.dim() == 3, "row [B, T, columns]");
  ChunkAttnParams p = chunk_sizes(row.size(0), row.size(1), H, G, dim, vdim, 0, 1.0);
  chunk_row(p, row, bias, q_w, k_w, rot, v_off, eps, cos_t, sin_t);
  TORCH_CHECK(base >= 0 && (rot == 0 || base + p.T <= p.npos), "positions exceed the rotary table");
  p.kv_start = starts(kv_start, row, p.B);
  p.base = base;
  p.rows = 1;
  c10::hip::HIPGuardMasqueradingAsCUDA guard(row.device());
  auto q = at::empty({p.B, p.T, H, dim}, row.options()), k = at::empty({p.B, p.T, G, dim}, row.options());
  auto v = at::empty({p.B, p.T, G, vdim}, row.options());
  p.q = q.data_ptr();
  p.k = k.data_ptr();
  p.v = v.data_ptr();
  launch_chunk_prepare(bf, p, false, cur_stream(row));
  return {q, k, v};
}

void chunk_kv(ChunkAttnParams& p, const at::Tensor& k, const at::Tensor& v) {
  p.k = k.data_ptr();
  p.v = v.data_ptr();
}

at::Tensor chunk_prefill(const at::Tensor& q, const at::Tensor& k, const at::Tensor& v, const at::Tensor& kc, const at::Tensor& vc,
                         int64_t chunk, double scale, const OptT& kv_start, int64_t base) {
  const bool bf = elem(q, "q");
  like(k, q, "k");
  like(v, q, "v");
  TORCH_CHECK(q.dim() == 4 && k.dim() == 4 && v.dim() == 4 && q.is_contiguous() && k.is_contiguous() && v.is_contiguous() &&
                  k.sizes() == at::IntArrayRef({q.size(0), q.size(1), k.size(2), q.size(3)}) &&
                  v.sizes() == at::IntArrayRef({q.size(0), q.size(1), k.size(2), v.size(3)}),
              "q [B, T, H, dim], k [B, T, G, dim], v [B, T, G, vdim] contiguous");
  ChunkAttnParams p = chunk_sizes(q.size(0), q.size(1), q.size(2), k.size(2), q.size(3), v.size(3), chunk, scale);
  chunk_cache(p, kc, vc, q);
  // every earlier position of the portion's first chunk has a row
  TORCH_CHECK(base >= 0 && base + p.T < kNoChunks && std::min<int64_t>(base, p.chunk) <= p.rows, "chunk_prefill: cache rows");
  chunk_kv(p, k, v);
  p.q = q.data_ptr();
  p.kv_start = starts(kv_start, q, p.B);
  p.base = base;
  c10::hip::HIPGuardMasqueradingAsCUDA guard(q.device());
  auto o = at::empty({p.B, p.T, static_cast<int64_t>(p.H) * p.vdim}, q.options());
  p.o = o.data_ptr();
  if (bf && chunk_prefill_mfma_ok(p)) launch_chunk_prefill_mfma(p, cur_stream(q));
  else launch_chunk_prefill_any(bf, p, cur_stream(q));
  return o;
}

void chunk_store(const at::Tensor& k, const at::Tensor& v, at::Tensor kc, at::Tensor vc, int64_t chunk, const OptT& kv_start,
                 int64_t base) {
  const bool bf = elem(k, "k");
  like(v, k, "v");
  TORCH_CHECK(k.dim() == 4 && v.dim() == 4 && k.is_contiguous() && v.is_contiguous() &&
                  v.sizes() == at::IntArrayRef({k.size(0), k.size(1), k.size(2), v.size(3)}),
              "k [B, T, G, dim], v [B, T, G, vdim] contiguous");
  ChunkAttnParams p = chunk_sizes(k.size(0), k.size(1), k.size(2), k.size(2), k.size(3), v.size(3), chunk, 1.0);
  chunk_cache(p, kc, vc, k);
  TORCH_CHECK(base >= 0 && std::min<int64_t>(base + p.T, p.chunk) <= p.rows, "chunk_store: cache rows");
  chunk_kv(p, k, v);
  p.kv_start = starts(kv_start, k, p.B);
  p.base = base;
  c10::hip::HIPGuardMasqueradingAsCUDA guard(k.device());
  launch_chunk_store(bf, p, cur_stream(k));
}

at::Tensor chunk_decode(const at::Tensor& row, const at::Tensor& bias, const at::Tensor& q_w, const at::Tensor& k_w, int64_t H,
                        int64_t G, int64_t dim, int64_t vdim, int64_t rot, int64_t v_off, double eps, at::Tensor kc,
                        at::Tensor vc, int64_t chunk, double scale, const at::Tensor& slot, const OptT& kv_start,
                        const at::Tensor& cos_t, const at::Tensor& sin_t) {
  const bool bf = elem(row, "row");
  TORCH_CHECK(row.dim() == 3 && row.size(1) == 1, "row [B, 1, columns]");
  ChunkAttnParams p = chunk_sizes(row.size(0), 1, H, G, dim, vdim, chunk, scale);
  chunk_row(p, row, bias, q_w, k_w, rot, v_off, eps, cos_t, sin_t);
  chunk_cache(p, kc, vc, row);
  p.kv_start = starts(kv_start, row, p.B);
  p.slot = slot_ptr(slot, row);
  // enough key splits to fill the chip, none shorter than a step of the fullest cache
  const int64_t groups = static_cast<int64_t>(p.B) * G * ((H / G + 15) / 16);
  int64_t ns = std::min<int64_t>((512 + groups - 1) / groups, (p.rows + 127) / 128);
  p.ns = static_cast<int>(std::max<int64_t>(1, std::min<int64_t>(ns, 256)));
  c10::hip::HIPGuardMasqueradingAsCUDA guard(row.device());
  auto q = at::empty({p.B, 1, H, dim}, row.options()), o = at::empty({p.B, 1, H * vdim}, row.options());
  p.q = q.data_ptr();
  p.k = p.v = nullptr;
  p.o = o.data_ptr();
  at::Tensor po, ml;
  if (p.ns > 1) {
    po = at::empty({p.B, H, p.ns, vdim}, row.options().dtype(at::kFloat));
    ml = at::empty({p.B, H, p.ns, 2}, po.options());
    p.part_o = po.data_ptr<float>();
    p.part_ml = ml.data_ptr<float>();
  }
  launch_chunk_prepare(bf, p, true, cur_stream(row));
  launch_chunk_decode(bf, p, cur_stream(row));
  return o;
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
  m.def("stream_gemm_post(Tensor a, Tensor w, Tensor(a!) x, float alpha, Tensor? bias, Tensor? res_ssq, Tensor? res_w, Tensor norm_w, float eps) -> (Tensor, Tensor)");
  m.def("stream_gemm_cap(Tensor a, Tensor w, float cap) -> Tensor");
  m.def("relu2(Tensor u) -> Tensor");
  m.def("post_norm(Tensor(a!) x, Tensor? delta, Tensor? bias, float alpha, Tensor w, Tensor? w2, float eps, bool bf16) -> Tensor");
  m.def("geglu(Tensor u) -> Tensor");
  m.def("softcap(Tensor z, float cap) -> Tensor");
  m.def("lru_prefill(Tensor yx, Tensor bias, Tensor conv_w, Tensor conv_b, Tensor gates, Tensor gates_b, Tensor lam, float c, Tensor(a!) state, Tensor(b!) hist, Tensor? kv_start, int base) -> Tensor");
  m.def("lru_decode(Tensor yx, Tensor bias, Tensor conv_w, Tensor conv_b, Tensor gates, Tensor gates_b, Tensor lam, float c, Tensor(a!) state, Tensor(b!) hist, Tensor slot, Tensor? kv_start) -> Tensor");
  m.def("gla_prefill(Tensor proj, Tensor a2, Tensor a2_b, Tensor norm_w, int H, int dim, int vdim, float tau, float eps, Tensor(a!) state, Tensor? kv_start, int base) -> Tensor");
  m.def("gla_decode(Tensor proj, Tensor a2, Tensor a2_b, Tensor norm_w, int H, int dim, int vdim, float tau, float eps, Tensor(a!) state, Tensor(b!)? cnt) -> Tensor");
  m.def("chunk_prepare(Tensor row, Tensor bias, Tensor q_w, Tensor k_w, int H, int G, int dim, int vdim, int rot, int v_off, float eps, Tensor? kv_start, Tensor cos, Tensor sin, int base) -> (Tensor, Tensor, Tensor)");
  m.def("chunk_prefill(Tensor q, Tensor k, Tensor v, Tensor kc, Tensor vc, int chunk, float scale, Tensor? kv_start, int base) -> Tensor");
  m.def("chunk_store(Tensor k, Tensor v, Tensor(a!) kc, Tensor(b!) vc, int chunk, Tensor? kv_start, int base) -> ()");
  m.def("chunk_decode(Tensor row, Tensor bias, Tensor q_w, Tensor k_w, int H, int G, int dim, int vdim, int rot, int v_off, float eps, Tensor(a!) kc, Tensor(b!) vc, int chunk, float scale, Tensor slot, Tensor? kv_start, Tensor cos, Tensor sin) -> Tensor");
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
  m.impl("stream_gemm_post", &dla::stream_gemm_post);
  m.impl("stream_gemm_cap", &dla::stream_gemm_cap);
  m.impl("relu2", &dla::relu2);
  m.impl("post_norm", &dla::post_norm);
  m.impl("geglu", &dla::geglu);
  m.impl("softcap", &dla::softcap);
  m.impl("lru_prefill", &dla::lru_prefill);
  m.impl("lru_decode", &dla::lru_decode);
  m.impl("gla_prefill", &dla::gla_prefill);
  m.impl("gla_decode", &dla::gla_decode);
  m.impl("chunk_prepare", &dla::chunk_prepare);
  m.impl("chunk_prefill", &dla::chunk_prefill);
  m.impl("chunk_store", &dla::chunk_store);
  m.impl("chunk_decode", &dla::chunk_decode);
  m.impl("retention_prefill", &dla::retention_prefill);
  m.impl("retention_decode", &dla::retention_decode);
  m.impl("latent_prepare", &dla::latent_prepare);
  m.impl("latent_prefill", &dla::latent_prefill);
  m.impl("latent_decode", &dla::latent_decode);
}
