"""Ops on the fp32 residual stream of per-layer designs (models/mixers.py).

The stream x stays fp32 in HBM; matrix products read it normed (or just cast) to the compute dtype.
One kernel per visit (csrc/mix/stream.hip): add the pending update (optionally RMS-normed first, and
optionally with the embedding output re-injected), write x back, write the normed rows. bf16 and
fp32 compute dtypes run the same kernels. CPU tensors use the PyTorch forms below.
"""
from __future__ import annotations

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


def stream_linear(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x W^T in the compute dtype (fp32: true fp32 products)."""
    return F.linear(x, w)


def head_logits(h: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    return F.linear(h, w)
