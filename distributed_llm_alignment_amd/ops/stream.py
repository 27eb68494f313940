"""Ops on the fp32 residual stream of per-layer designs (models/mixers.py).

The stream x stays fp32 in HBM; matrix products read it normed (or just cast) to the compute dtype.
One kernel per visit (csrc/mix/stream.hip): add the pending update (optionally RMS-normed first, and
optionally with the embedding output re-injected), write x back, write the normed rows. bf16 and
fp32 compute dtypes run the same kernels. CPU tensors use the PyTorch forms below.
"""
from __future__ import annotations

import os
from typing import Optional, Tuple

import torch
import torch.nn.functional as F

from . import _ext
from .embedding import _bad_word


def embed_stream(ids: torch.Tensor, table: torch.Tensor, scale: float) -> torch.Tensor:
    """fp32 [.., H] = table[ids] * scale (out-of-range ids: zero rows + the embedding error word,
    see ops.embedding.check_ids)."""
    if _ext.use_native(table):
        return _ext.require("mix").embed_stream(ids.contiguous(), table, float(scale), _bad_word(table.device))
    return F.embedding(ids, table).float() * scale


def _rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def stream_norm(x: torch.Tensor, delta: Optional[torch.Tensor], delta_w: Optional[torch.Tensor],
                inject: Optional[torch.Tensor], w: Optional[torch.Tensor], eps: float, offset: float,
                dtype: torch.dtype) -> Tuple[torch.Tensor, torch.Tensor]:
    """x += delta (RMS-normed and weighted by delta_w when given) + inject, then
    y = RMSNorm(x) * (offset + w) in `dtype` (w None: y = x in `dtype`). Returns (y, x); the GPU
    kernel updates x in place."""
    if _ext.use_native(x):
        y = _ext.require("mix").stream_norm(x, delta, delta_w, inject, w, float(eps), float(offset),
                                            dtype == torch.bfloat16)
        return y, x
    if delta is not None:
        d = delta.float()
        x = x + (d if delta_w is None else _rms(d, eps) * delta_w.float())
    if inject is not None:
        x = x + inject
    y = x if w is None else _rms(x, eps) * (offset + w.float())
    return y.to(dtype), x


def post_norm(x: torch.Tensor, delta: Optional[torch.Tensor], bias: Optional[torch.Tensor], alpha: float, w: torch.Tensor,
              w2: Optional[torch.Tensor], eps: float, dtype: torch.dtype) -> Tuple[torch.Tensor, torch.Tensor]:
    """Norm after the sum: x <- RMSNorm(alpha x + delta + bias) * w (fp32); y = x, or RMSNorm(x) * w2
    when w2 is given (the model's last norm), in `dtype`. Returns (y, x); the GPU kernel updates x in
    place."""
    if _ext.use_native(x):
        y = _ext.require("mix").post_norm(x, delta, bias, float(alpha), w, w2, float(eps), dtype == torch.bfloat16)
        return y, x
    s = alpha * x if delta is None else alpha * x + delta.float()
    if bias is not None:
        s = s + bias.float()
    x = _rms(s, eps) * w.float()
    return (x if w2 is None else _rms(x, eps) * w2.float()).to(dtype), x


def side_gate(z: torch.Tensor, ids: torch.Tensor, side_embed: torch.Tensor, off: int) -> torch.Tensor:
    """gelu_tanh(z) * side_embed[ids, off : off + z.shape[-1]]."""
    if _ext.use_native(z):
        return _ext.require("mix").side_gate(z, ids.contiguous(), side_embed, int(off))
    e = F.embedding(ids, side_embed[:, off:off + z.shape[-1]])
    return (F.gelu(z.float(), approximate="tanh") * e.float()).to(z.dtype)


def relu2(u: torch.Tensor) -> torch.Tensor:
    """relu(u)^2."""
    if _ext.use_native(u):
        if torch.is_grad_enabled() and u.requires_grad:
            raise NotImplementedError("relu2 on the GPU is inference only")
        return _ext.require("mix").relu2(u)
    return torch.relu(u.float()).square().to(u.dtype)


def geglu(u: torch.Tensor) -> torch.Tensor:
    """u [.., 2 F] = [gate | up] -> gelu_tanh(gate) * up."""
    if _ext.use_native(u):
        if torch.is_grad_enabled() and u.requires_grad:
            raise NotImplementedError("geglu on the GPU is inference only")
        return _ext.require("mix").geglu(u)
    gate, up = u.float().chunk(2, -1)
    return (F.gelu(gate, approximate="tanh") * up).to(u.dtype)


def softcap(z: torch.Tensor, cap: float) -> torch.Tensor:
    """cap * tanh(z / cap), fp32."""
    if _ext.use_native(z):
        return _ext.require("mix").softcap(z, float(cap))
    return cap * torch.tanh(z.float() / cap)


def stream_linear(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x W^T in the compute dtype (fp32: true fp32 products)."""
    return F.linear(x, w)


def head_logits(h: torch.Tensor, w: torch.Tensor, cap: float = 0.0) -> torch.Tensor:
    """h w^T, with a soft cap cap * tanh(. / cap) in fp32."""
    rows = h.numel() // h.shape[-1]
    if h.is_cuda and fused_ok(rows, h.dtype, w) and not torch.is_grad_enabled():
        if cap:
            return _ext.require("mix").stream_gemm_cap(_rows(h), w, float(cap)).view(*h.shape[:-1], w.shape[0])
        return fused_linear(h, w)
    z = F.linear(h, w)
    return softcap(z, cap) if cap else z


# ------------------------------------------------------------------------ fused decode projections
# (csrc/mix/stream_gemm.hip) few rows: the norm before a projection and the stream add / activation /
# gate behind it run inside the projection's launch. DLA_STREAM_FUSED=0: library GEMMs + the kernels above.
STREAM_FUSED = os.environ.get("DLA_STREAM_FUSED", "1") != "0"
# (17 .. 32 rows run too, but every workgroup re-reads all of a for its 16 columns: at 32 rows that is
# more L2 traffic than the weights, and the library's GEMMs are ahead)
STREAM_FUSED_ROWS = int(os.environ.get("DLA_STREAM_FUSED_ROWS", "16"))
_STORE, _RELU2, _GATE, _STREAM, _GEGLU = 0, 1, 2, 3, 5  # (4, 6: ops of their own)


def fused_ok(rows: int, dtype: torch.dtype, *weights: torch.Tensor) -> bool:
    """These projections can run on the fused decode kernel (bf16, GPU, <= 32 rows, K % 8 == 0)."""
    return (STREAM_FUSED and 1 <= rows <= min(STREAM_FUSED_ROWS, 32) and dtype == torch.bfloat16
            and all(w.is_cuda and w.dim() == 2 and w.is_contiguous() and w.shape[1] % 8 == 0 and w.data_ptr() % 16 == 0
                    for w in weights))


def _rows(a: torch.Tensor) -> torch.Tensor:
    return a.reshape(-1, a.shape[-1]).contiguous()


def fused_linear(a: torch.Tensor, w: torch.Tensor, ssq: Optional[torch.Tensor] = None, eps: float = 0.0,
                 relu2: bool = False) -> torch.Tensor:
    """rowscale * (a W^T) [then relu(.)^2]; `ssq`: partial sums of squares from `fused_add` (rowscale =
    rsqrt(mean + eps)), None: no scale."""
    y, _ = _ext.require("mix").stream_gemm(_rows(a), w, _RELU2 if relu2 else _STORE, ssq, float(eps), None, None, 0.0,
                                           None, None, 0)
    return y.view(*a.shape[:-1], w.shape[0])


def fused_geglu(a: torch.Tensor, w: torch.Tensor, ssq: Optional[torch.Tensor] = None, eps: float = 0.0) -> torch.Tensor:
    """geglu(rowscale * (a W^T)), W = [gate; up]."""
    y, _ = _ext.require("mix").stream_gemm(_rows(a), w, _GEGLU, ssq, float(eps), None, None, 0.0, None, None, 0)
    return y.view(*a.shape[:-1], w.shape[0] // 2)


def fused_post(a: torch.Tensor, w: torch.Tensor, x: torch.Tensor, alpha: float, bias: Optional[torch.Tensor],
               res_ssq: Optional[torch.Tensor], res_w: Optional[torch.Tensor], norm_w: torch.Tensor, eps: float):
    """x <- alpha x_prev + a W^T + bias (fp32, in place), x_prev = x or, with `res_ssq` (x's partial sums of
    squares) and `res_w`, RMSNorm(x) * res_w. Returns (x * norm_w in bf16, x's partial sums of squares):
    the next projection sees RMSNorm(x) * norm_w through its row scale."""
    y, ssq = _ext.require("mix").stream_gemm_post(_rows(a), w, x, float(alpha), bias, res_ssq, res_w, norm_w, float(eps))
    return y.view(*a.shape[:-1], w.shape[0]), ssq


def fused_gate(a: torch.Tensor, w: torch.Tensor, ids: torch.Tensor, side_embed: torch.Tensor, off: int) -> torch.Tensor:
    """side_gate(a W^T, ids, side_embed, off)."""
    y, _ = _ext.require("mix").stream_gemm(_rows(a), w, _GATE, None, 0.0, None, None, 0.0, ids.contiguous(), side_embed,
                                           int(off))
    return y.view(*a.shape[:-1], w.shape[0])


def fused_add(a: torch.Tensor, w: torch.Tensor, x: torch.Tensor, norm_w: Optional[torch.Tensor], offset: float):
    """x += a W^T (fp32, in place). Returns (x * (offset + norm_w), or x, in bf16; x's partial sums of
    squares): what the next projection needs to see RMSNorm(x)."""
    y, ssq = _ext.require("mix").stream_gemm(_rows(a), w, _STREAM, None, 0.0, x, norm_w, float(offset), None, None, 0)
    return y.view(*a.shape[:-1], w.shape[0]), ssq
