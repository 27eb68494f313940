"""Softmax attention whose keys are seen in chunks of the sequence: position i sees the positions
j <= i of its own chunk (chunk 0: one chunk of any length).

  prepare   biases, RMS norm of q and of k over their whole projections, rotary positions on the first
            `rot` dimensions of each head; the values are columns of the same projected row, biased
            only (with v_off = the keys' offset: the keys as projected)
  prefill   flash attention over the portion's own keys and, for the portion's first chunk, the
            cached ones (csrc/mix/chunk_prefill.hip; any sizes and fp32: csrc/mix/chunk_attn.hip)
  store     the last chunk's keys and values into the cache
  decode    split-key attention on the cache

The cache holds one chunk per sequence, [B, kv_heads, rows, dim]: position p sits in row p % chunk, so
rows 0 .. p % chunk are exactly what position p sees, whatever the rows behind them still hold. A
token's position is its column minus kv_start[b]; columns below kv_start[b] are padding.
"""
from __future__ import annotations

from typing import NamedTuple, Tuple

import torch

from . import _ext
from .latent import _positions, _rotate
from .stream import _rms


class Heads(NamedTuple):
    """Sizes and constants of one attention mixer."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    rot: int
    v_off: int     # column of the values in a projected row
    chunk: int     # 0: no chunks
    scale: float
    eps: float


def _prepared(row, bias, q_w, k_w, h: Heads, cos, sin, pos):
    B, T, _ = row.shape
    x = row.float() + bias.float()
    nq, nk = h.heads * h.dim, h.kv_heads * h.dim
    q = (_rms(x[..., :nq], h.eps) * q_w.float()).view(B, T, h.heads, h.dim)
    k = (_rms(x[..., nq:nq + nk], h.eps) * k_w.float()).view(B, T, h.kv_heads, h.dim)
    v = x[..., h.v_off:h.v_off + h.kv_heads * h.vdim].reshape(B, T, h.kv_heads, h.vdim)
    if h.rot:
        q, k = (torch.cat([_rotate(t[..., :h.rot], cos, sin, pos), t[..., h.rot:]], -1) for t in (q, k))
    return q.to(row.dtype), k.to(row.dtype), v.to(row.dtype)


def prepare(row, bias, q_w, k_w, h: Heads, kv_start, cos, sin, base: int) -> Tuple[torch.Tensor, ...]:
    """row [B, T, columns] (no bias yet) -> q [B, T, heads, dim], k [B, T, kv_heads, dim], v."""
    if _ext.use_native(row):
        return _ext.require("mix").chunk_prepare(row, bias, q_w, k_w, *h[:6], h.eps, kv_start, cos, sin, int(base))
    return _prepared(row, bias, q_w, k_w, h, cos, sin, _positions(row.shape[0], row.shape[1], base, kv_start, row.device))


def _attend(q, k, v, h: Heads, qpos, kpos):
    """q [B, T, H, d], k / v [B, S, G, .], qpos [B, T], kpos [B, S] (< 0: not there)."""
    g = h.heads // h.kv_heads
    kf, vf = (t.float().repeat_interleave(g, 2) for t in (k, v))
    i, j = qpos.unsqueeze(2), kpos.unsqueeze(1)
    ok = (j >= 0) & (j <= i)
    if h.chunk:
        ok = ok & (i.div(h.chunk, rounding_mode="floor") == j.div(h.chunk, rounding_mode="floor"))
    s = torch.einsum("bthd,bshd->bhts", q.float(), kf) * h.scale
    p = torch.nan_to_num(torch.softmax(s.masked_fill(~ok.unsqueeze(1), float("-inf")), -1))
    return torch.einsum("bhts,bshd->bthd", p, vf).to(q.dtype)


def _cached(kc, vc, h: Heads, pos):
    """The cached rows that position pos [B] (the next token's) sees, as (k, v [B, S, G, .], kpos)."""
    at = torch.arange(kc.shape[2], device=kc.device).expand(kc.shape[0], -1)
    pos = pos.clamp(min=0).view(-1, 1)
    first = pos.div(h.chunk, rounding_mode="floor") * h.chunk if h.chunk else torch.zeros_like(pos)
    kpos = torch.where(first + at < pos, first + at, torch.full_like(at, -1))
    return kc.transpose(1, 2), vc.transpose(1, 2), kpos


def _pos(B: int, T: int, base: int, kv_start, device):
    t = torch.arange(base, base + T, device=device).expand(B, T)
    return t if kv_start is None else t - kv_start.long().view(B, 1)


def prefill(q, k, v, kc, vc, h: Heads, kv_start, base: int) -> torch.Tensor:
    """A portion of T tokens per row at columns base .. : -> [B, T, heads * vdim]."""
    if _ext.use_native(q):
        return _ext.require("mix").chunk_prefill(q, k, v, kc, vc, h.chunk, h.scale, kv_start, int(base))
    B, T = q.shape[:2]
    pos = _pos(B, T, base, kv_start, q.device)
    ck, cv, cpos = _cached(kc, vc, h, pos[:, 0])
    if not base:
        cpos = torch.full_like(cpos, -1)
    o = _attend(q, torch.cat([ck, k], 1), torch.cat([cv, v], 1), h, pos, torch.cat([cpos, pos], 1))
    return o.reshape(B, T, h.heads * h.vdim)


def store(k, v, kc, vc, h: Heads, kv_start, base: int) -> None:
    """Write the portion's tokens that belong to the last token's chunk into the cache."""
    if _ext.use_native(k):
        _ext.require("mix").chunk_store(k, v, kc, vc, h.chunk, kv_start, int(base))
        return
    B, T = k.shape[:2]
    pos = _pos(B, T, base, kv_start, k.device)
    c = h.chunk or 1 << 40
    for b in range(B):
        keep = (pos[b] >= 0) & (pos[b] // c == pos[b, -1] // c)
        kc[b, :, pos[b, keep] % c] = k[b, keep].transpose(0, 1)
        vc[b, :, pos[b, keep] % c] = v[b, keep].transpose(0, 1)


def decode(row, bias, q_w, k_w, kc, vc, h: Heads, slot, kv_start, cos, sin, base: int) -> torch.Tensor:
    """One new token per row at column `base` (`slot` on the device): prepare, cache write and
    attention. row [B, 1, columns] -> [B, 1, heads * vdim]."""
    if _ext.use_native(row):
        return _ext.require("mix").chunk_decode(row, bias, q_w, k_w, *h[:6], h.eps, kc, vc, h.chunk, h.scale, slot,
                                                kv_start, cos, sin)
    B = row.shape[0]
    q, k, v = prepare(row, bias, q_w, k_w, h, kv_start, cos, sin, base)
    pos = _pos(B, 1, base, kv_start, row.device)
    store(k, v, kc, vc, h, kv_start, base)
    ck, cv, cpos = _cached(kc, vc, h, pos[:, 0])
    at = pos % h.chunk if h.chunk else pos
    cpos = cpos.scatter(1, at, pos)
    return _attend(q, ck, cv, h, pos, cpos).reshape(B, 1, h.heads * h.vdim)
