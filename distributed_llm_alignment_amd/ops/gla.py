"""Gated linear attention: linear attention whose state decays per key channel and token.

    z = a2 (a1 h) + b,   log alpha = log sigmoid(z) / tau
    S_t = diag(alpha_t) S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t dim^(-1/2)
    y = rms(o) * w * silu(g)      per head (w shared by the heads)

`proj` rows are [q (H dim) | k (H dim) | v (H vdim) | g (H vdim) | a1 h (rank)]; the second product of the
decay, the decays, the state and the norm are fp32. Columns below kv_start[b] are padding (they add
nothing to the state). The state is kept transposed, [B, H, vdim, dim].

prefill (csrc/mix/gla_mfma.hip, bf16): chunks as in ops.retention, with every product of decays
written so that no factor exceeds one; other sizes and fp32 run the recurrence (csrc/mix/gla.hip), as
decode does.
"""
from __future__ import annotations

import torch
import torch.nn.functional as F

from . import _ext
from .retention import _counters
from .stream import _rms


def prefill(proj, a2, a2_b, norm_w, H: int, dim: int, vdim: int, tau: float, eps: float, state, slot, kv_start,
            base: int) -> torch.Tensor:
    """T tokens per row after `base` earlier columns (0: the state starts at zero, whatever it holds);
    state [B, H, vdim, dim] fp32 is advanced in place. -> [B, T, H * vdim]."""
    if _ext.use_native(proj):
        return _ext.require("mix").gla_prefill(proj, a2, a2_b, norm_w, H, dim, vdim, float(tau), float(eps), state,
                                               kv_start, int(base))
    B, T, _ = proj.shape
    q, k, v, g, a = proj.float().split([H * dim, H * dim, H * vdim, H * vdim, a2.shape[1]], -1)
    la = F.logsigmoid(F.linear(a, a2.float(), a2_b.float())).view(B, T, H, dim) / tau
    q, k, v = q.view(B, T, H, dim) * dim ** -0.5, k.view(B, T, H, dim), v.view(B, T, H, vdim)
    if kv_start is not None:
        real = (torch.arange(base, base + T) >= kv_start.long().view(-1, 1)).view(B, T, 1, 1)
        k, v, la = (torch.where(real, t, torch.zeros_like(t)) for t in (k, v, la))
    S = state.clone() if base else torch.zeros_like(state)
    out = []
    for t in range(T):
        S = la[:, t].exp().unsqueeze(2) * S + v[:, t].unsqueeze(3) * k[:, t].unsqueeze(2)
        out.append((S * q[:, t].unsqueeze(2)).sum(-1))
    state.copy_(S)
    o = _rms(torch.stack(out, 1), eps) * norm_w.float()
    return (o.reshape(B, T, H * vdim) * F.silu(g)).to(proj.dtype)


def decode(proj, a2, a2_b, norm_w, H: int, dim: int, vdim: int, tau: float, eps: float, state, slot, kv_start,
           base: int) -> torch.Tensor:
    """One new token per row."""
    if _ext.use_native(proj):
        return _ext.require("mix").gla_decode(proj, a2, a2_b, norm_w, H, dim, vdim, float(tau), float(eps), state,
                                              _counters(proj.device, proj.shape[0] * H))
    return prefill(proj, a2, a2_b, norm_w, H, dim, vdim, tau, eps, state, slot, kv_start, base)
