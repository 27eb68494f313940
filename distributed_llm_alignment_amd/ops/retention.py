"""Retention: linear attention with one fixed decay per head and no denominator.

    S_t = decay S_(t-1) + k_t v_t^T,  o_t = S_t^T q_t,  y = (o / rms(o)) * silu(g)   per head

prefill runs it in chunks (csrc/mix/retention.hip: each chunk's own state in parallel, a scan over
the chunks, then every chunk's outputs from its start state and its own tokens); decode is one pass
over the state per token. State, decays, rotated keys and the per-head norm are fp32.
`qkvg` rows are [q (H * dim) | k (H * dim) | v (H * vdim) | g (H * vdim)]; columns below kv_start[b]
are padding (they add nothing to the state); `decay` is [2, H] = (decay, log2 decay).
"""
from __future__ import annotations

import torch

from . import _ext
from .latent import _positions
from .stream import _rms


_COUNTERS = {}  # per device: arrival counters of the split decode (zero between launches)


def _counters(device, n: int):
    c = _COUNTERS.get(device)
    if c is None or c.numel() < n:
        if torch.cuda.is_current_stream_capturing():
            return None  # never allocated (zeroed) inside a captured graph
        if c is not None:  # an outgrown tensor stays alive: captured decode steps keep using it
            _COUNTERS.setdefault("outgrown", []).append(c)
        c = _COUNTERS[device] = torch.zeros(max(1024, n), dtype=torch.int32, device=device)
    return c


def _rotated(x, rot, cos, sin, pos):
    half = rot // 2
    c, s = cos[pos].unsqueeze(2), sin[pos].unsqueeze(2)
    u, v = x[..., :half], x[..., half:rot]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., rot:]], -1)


def prefill(qkvg, H: int, dim: int, vdim: int, rot: int, eps: float, decay, state, slot, kv_start, cos, sin,
            base: int) -> torch.Tensor:
    """T tokens per row after `base` earlier columns (0: the state starts at zero, whatever it holds);
    state [B, H, vdim, dim] fp32 (transposed: one
    output column's row is contiguous) is advanced in place. -> [B, T, H * vdim]."""
    if _ext.use_native(qkvg):
        return _ext.require("mix").retention_prefill(qkvg, H, dim, vdim, rot, float(eps), decay, state, kv_start,
                                                     cos, sin, int(base))
    B, T, _ = qkvg.shape
    q, k, v, g = qkvg.float().split([H * dim, H * dim, H * vdim, H * vdim], -1)
    pos = _positions(B, T, base, kv_start, qkvg.device)
    q = _rotated(q.view(B, T, H, dim), rot, cos, sin, pos)
    k = _rotated(k.view(B, T, H, dim), rot, cos, sin, pos) * dim ** -0.5
    v = v.view(B, T, H, vdim)
    t = torch.arange(T, device=qkvg.device)
    if kv_start is not None:
        k = k * (t.view(1, T) + base >= kv_start.view(B, 1)).view(B, T, 1, 1)
    S0 = state.clone() if base > 0 else torch.zeros_like(state)
    l2 = decay[1].view(H, 1, 1)
    w = torch.exp2((t.view(T, 1) - t).clamp(min=0) * l2) * (t.view(T, 1) >= t)
    o = torch.einsum("bthd,bshd->bhts", q, k) * w
    o = torch.einsum("bhts,bshv->bthv", o, v)
    o = o + torch.einsum("bthd,bhvd->bthv", q * torch.exp2((t + 1).view(1, T, 1, 1) * decay[1].view(1, 1, H, 1)), S0)
    tail = torch.exp2((T - 1 - t).view(1, T, 1, 1) * decay[1].view(1, 1, H, 1))
    state.copy_(torch.exp2(T * l2) * S0 + torch.einsum("bthd,bthv->bhvd", k * tail, v))
    return (_rms(o, eps).reshape(B, T, H * vdim) * torch.nn.functional.silu(g)).to(qkvg.dtype)


def decode(qkvg, H: int, dim: int, vdim: int, rot: int, eps: float, decay, state, slot, kv_start, cos, sin,
           base: int) -> torch.Tensor:
    """One new token per row (column `base`, on the device in `slot`)."""
    if _ext.use_native(qkvg):
        return _ext.require("mix").retention_decode(qkvg, H, dim, vdim, rot, float(eps), decay, state, slot,
                                                    kv_start, cos, sin, _counters(qkvg.device, qkvg.shape[0] * H))
    return prefill(qkvg, H, dim, vdim, rot, eps, decay, state, slot, kv_start, cos, sin, base)
