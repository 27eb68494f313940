"""Latent attention: keys and values are projections of one cached latent per token, plus one rotated
key part shared by all heads; softmax over a sliding window.

  prepare   both latents' RMS norms, the shared key part's rotation, the cache write   (one kernel)
  prefill   flash attention over up-projected keys and values; the query's rotated part is rotated
            as it is loaded (csrc/mix/latent_prefill.hip)
  decode    "absorbed" form: the query is taken into latent space (q W_uk), scores and the weighted
            sum run against the latent cache itself (one read for all heads), and the result goes
            through W_uv (csrc/mix/latent_decode.hip)

Cache rows are [latent (kv_rank) | rotated key part (rot)], [B, T_max, kv_rank + rot]. Columns
below kv_start[b] are padding; a token's position is its column minus kv_start[b].
"""
from __future__ import annotations

from typing import Optional

import torch

from . import _ext
from .stream import _rms


def _positions(B: int, T: int, base: int, kv_start, device) -> torch.Tensor:
    t = torch.arange(base, base + T, device=device).expand(B, T)
    return t if kv_start is None else (t - kv_start.long().view(B, 1)).clamp(min=0)


def _rotate(x: torch.Tensor, cos, sin, pos) -> torch.Tensor:
    """x [B, T, H, rot] fp32, rotate-half over all of it."""
    half = x.shape[-1] // 2
    c, s = cos[pos].unsqueeze(2), sin[pos].unsqueeze(2)
    u, v = x[..., :half], x[..., half:]
    return torch.cat([u * c - v * s, v * c + u * s], -1)


def prepare(down, q_norm_w, kv_norm_w, eps, latent, slot, kv_start, cos, sin, base: int) -> torch.Tensor:
    """down [B, T, q_rank + kv_rank + rot] -> normed query latent [B, T, q_rank]; columns
    base .. base + T - 1 of the cache get the normed latent and the rotated key part (`slot`: base on
    the device, what the GPU kernel reads)."""
    if _ext.use_native(down):
        return _ext.require("mix").latent_prepare(down, q_norm_w, kv_norm_w, float(eps), latent, slot, kv_start,
                                                  cos, sin)
    B, T, _ = down.shape
    qr, R = q_norm_w.shape[0], kv_norm_w.shape[0]
    cq = (_rms(down[..., :qr].float(), eps) * q_norm_w.float()).to(down.dtype)
    c = _rms(down[..., qr:qr + R].float(), eps) * kv_norm_w.float()
    kr = _rotate(down[..., None, qr + R:].float(), cos, sin, _positions(B, T, base, kv_start, down.device))
    latent[:, base:base + T] = torch.cat([c, kr[:, :, 0]], -1).to(latent.dtype)
    return cq


def _weights(s: torch.Tensor, q_cols, k_cols, window: int, kv_start) -> torch.Tensor:
    """Softmax of s [B, H, Tq, Tk] over the visible columns (0 where a row sees none)."""
    i, j = q_cols.view(1, -1, 1), k_cols.view(1, 1, -1)
    ok = j <= i
    if window:
        ok = ok & (i - j < window)
    if kv_start is not None:
        ok = ok & (j >= kv_start.view(-1, 1, 1))
    return torch.nan_to_num(torch.softmax(s.masked_fill(~ok.unsqueeze(1), float("-inf")), -1))


def prefill(q, kv, kr, H: int, dim: int, rot: int, vdim: int, scale: float, window: int, kv_start, cos, sin,
            q_base: int, k_base: int) -> torch.Tensor:
    """q [B, T, H * (dim + rot)] (unrotated), kv [B, S, H * (dim + vdim)] = [keys | values], kr
    [B, S, rot]; query t sits at column q_base + t, key s at k_base + s. -> [B, T, H * vdim]."""
    if _ext.use_native(q):
        return _ext.require("mix").latent_prefill(q, kv, kr, H, dim, rot, vdim, float(scale), int(window), kv_start,
                                                  cos, sin, int(q_base), int(k_base))
    B, T, _ = q.shape
    S = kv.shape[1]
    qf = q.float().view(B, T, H, dim + rot)
    qr = _rotate(qf[..., dim:], cos, sin, _positions(B, T, q_base, kv_start, q.device))
    k = kv[..., :H * dim].float().view(B, S, H, dim)
    v = kv[..., H * dim:].float().view(B, S, H, vdim)
    s = torch.einsum("bthd,bshd->bhts", qf[..., :dim], k) + torch.einsum("bthd,bsd->bhts", qr, kr.float())
    ar = lambda n, b: torch.arange(b, b + n, device=q.device)  # noqa: E731
    p = _weights(s * scale, ar(T, q_base), ar(S, k_base), window, kv_start)
    return torch.einsum("bhts,bshd->bthd", p, v).reshape(B, T, H * vdim).to(q.dtype)


def decode(q, latent, kv_up, H: int, dim: int, rot: int, vdim: int, scale: float, window: int, slot, kv_start,
           cos, sin, base: int) -> torch.Tensor:
    """One new token per row, at column `base` (`slot` on the device): q [B, 1, H * (dim + rot)] ->
    [B, 1, H * vdim] against the latent cache."""
    if _ext.use_native(q):
        return _ext.require("mix").latent_decode(q, latent, kv_up, H, dim, rot, vdim, float(scale), int(window),
                                                 slot, kv_start, cos, sin)
    B, R = q.shape[0], kv_up.shape[1]
    qf = q.float().view(B, 1, H, dim + rot)
    qr = _rotate(qf[..., dim:], cos, sin, _positions(B, 1, base, kv_start, q.device))
    ql = torch.einsum("bthd,hdr->bthr", qf[..., :dim], kv_up[:H * dim].float().view(H, dim, R))
    seen = latent[:, :base + 1].float()
    s = torch.einsum("bthr,bsr->bhts", ql, seen[..., :R]) + torch.einsum("bthr,bsr->bhts", qr, seen[..., R:])
    ar = torch.arange(base + 1, device=q.device)
    p = _weights(s * scale, ar[base:], ar, window, kv_start)
    o = torch.einsum("bhts,bsr->bthr", p, seen[..., :R])
    o = torch.einsum("bthr,hdr->bthd", o, kv_up[H * dim:].float().view(H, vdim, R))
    return o.reshape(B, 1, H * vdim).to(q.dtype)
