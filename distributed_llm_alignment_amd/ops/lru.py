"""Real-gated linear recurrent unit behind a short causal convolution (Griffin's recurrent block).

    u_t = conv(x)_t                       depthwise, `taps` inputs, zeros before the start
    r_t, i_t = sigmoid(block-diagonal products of u_t)
    log a_t = -c r_t softplus(lam)        c = 8
    S_t = a_t S_(t-1) + sqrt(1 - a_t^2) i_t u_t
    out_t = S_t * gelu_tanh(y_t)

`yx` rows are [y (W) | x (W)] as projected, `bias` [2 W] is added here. Recurrence, gates and decays are
fp32. What a sequence carries: `state` [B, W] fp32, and `hist` [B, taps, W], the last projected x rows
without their bias in a ring (column c sits at c % taps, so a step writes no row that another part of
the step still reads). Columns below kv_start[b] are padding: they leave the state alone, and the
convolution sees zeros there.

prefill (csrc/mix/lru.hip): convolution, gates and each tile's scan in registers; a scan over the
tiles; start state, gelu gate and the store. decode: one launch.
"""
from __future__ import annotations

import torch
import torch.nn.functional as F

from . import _ext

DECAY = 8.0


def prefill(yx, bias, conv_w, conv_b, gates, gates_b, lam, state, hist, slot, kv_start, base: int) -> torch.Tensor:
    """T tokens per row after `base` earlier columns (0: state and history start empty, whatever they
    hold). gates [2 blocks, n, n] = the r gate's blocks, then the i gate's. -> [B, T, W]."""
    if _ext.use_native(yx):
        return _ext.require("mix").lru_prefill(yx, bias, conv_w, conv_b, gates, gates_b, lam, DECAY, state, hist,
                                               kv_start, int(base))
    B, T, _ = yx.shape
    W, taps = conv_w.shape
    nb, n = gates.shape[0] // 2, gates.shape[1]
    y, x = yx.float()[..., :W] + bias[:W].float(), yx[..., W:]
    pos = torch.arange(base, base + T) if kv_start is None else \
        torch.arange(base, base + T) - kv_start.long().view(-1, 1)
    pos = pos.expand(B, T)
    cols = torch.arange(base - taps + 1, base + T)
    before = hist[:, cols[:taps - 1] % taps] if base else torch.zeros_like(hist[:, :taps - 1])
    xs = torch.cat([before, x], 1).float() + bias[W:].float()
    seen = cols if kv_start is None else cols - kv_start.long().view(-1, 1)
    xs = xs.masked_fill(~(seen >= 0).expand(B, -1).unsqueeze(-1), 0.0)
    u = F.conv1d(xs.transpose(1, 2), conv_w.float().unsqueeze(1), conv_b.float(), groups=W).transpose(1, 2)
    u = u.to(yx.dtype).float()
    g = torch.einsum("btni,noi->btno", u.view(B, T, nb, n).repeat(1, 1, 2, 1), gates.float()) + gates_b.float()
    g = torch.sigmoid(g).reshape(B, T, 2, W)
    log_a = -DECAY * g[:, :, 0] * F.softplus(lam.float())
    b = torch.sqrt(-torch.expm1(2 * log_a)) * g[:, :, 1] * u
    real = (pos >= 0).unsqueeze(-1)
    a, b = torch.where(real, log_a.exp(), torch.ones_like(log_a)), torch.where(real, b, torch.zeros_like(b))
    S = state.clone() if base else torch.zeros_like(state)
    out = []
    for t in range(T):
        S = a[:, t] * S + b[:, t]
        out.append(S)
    state.copy_(S)
    for t in range(max(0, T - taps), T):
        hist[:, (base + t) % taps] = x[:, t].to(hist.dtype)
    return (torch.stack(out, 1) * F.gelu(y, approximate="tanh")).to(yx.dtype)


def decode(yx, bias, conv_w, conv_b, gates, gates_b, lam, state, hist, slot, kv_start, base: int) -> torch.Tensor:
    """One new token per row (column `base`, on the device in `slot`)."""
    if _ext.use_native(yx):
        return _ext.require("mix").lru_decode(yx, bias, conv_w, conv_b, gates, gates_b, lam, DECAY, state, hist, slot,
                                              kv_start)
    return prefill(yx, bias, conv_w, conv_b, gates, gates_b, lam, state, hist, slot, kv_start, base)
