"""Layers of per-layer designs (`ModelConfig.layer_specs`): latent attention, retention, real-gated
recurrence, gated linear attention and chunked attention mixers, feed-forwards, the per-layer token
input, and the layers that string them together on an fp32 residual stream: norm before each
sublayer (`StreamLayer`) or after each sum (`PostNormLayer`).

A `StreamLayer` never adds its own output to the stream: it hands the last projection's output on as
the *pending* update of a `Stream`, and the next norm kernel adds it while it reads the stream (one
pass: add, optional norm of the update, optional embedding re-injection, norm of the sum). A
`PostNormLayer` hands its update on in the same way, with the norm that belongs to the sum. Mixers
keep what they need of the past in a slot of `generation.KVCache` (`new_slot`); a layer that runs
several times per forward gets one slot per run.
"""
from __future__ import annotations

import dataclasses
import math
from typing import Dict, List, Optional

import torch
import torch.nn as nn

from .. import ops
from .config import ModelConfig
from .layer_spec import decay_rank, window


def _param(*shape, device=None, dtype=None) -> nn.Parameter:
    return nn.Parameter(torch.empty(*shape, device=device, dtype=dtype))


@dataclasses.dataclass
class PostNorm:
    """What the sum alpha x + delta + bias is normed with."""

    w: torch.Tensor
    alpha: float
    eps: float
    bias: Optional[torch.Tensor] = None


@dataclasses.dataclass
class Stream:
    """fp32 residual stream x [B, T, H] plus the update not added yet: x + norm?(delta) + inject, or with
    `post` norm(alpha x + delta + bias)."""

    x: torch.Tensor
    delta: Optional[torch.Tensor] = None
    delta_w: Optional[torch.Tensor] = None  # plain RMS norm of delta with this weight before the add
    inject: Optional[torch.Tensor] = None
    post: Optional[PostNorm] = None
    # fused decode: x is the sum before `post`, these its partial sums of squares and its rows x * post.w
    ssq: Optional[torch.Tensor] = None
    rows: Optional[torch.Tensor] = None

    def norm(self, w, eps: float, offset: float, dtype) -> torch.Tensor:
        """Fold the pending update into x and return the normed rows."""
        y, self.x = ops.stream_norm(self.x, self.delta, self.delta_w, self.inject, w, eps, offset, dtype)
        self.delta = self.delta_w = self.inject = None
        return y

    def cast(self, eps: float, dtype) -> torch.Tensor:
        """Fold the pending update into x and return x in the compute dtype."""
        if self.post is None:
            return self.norm(None, eps, 0.0, dtype)
        return self._post(None, dtype)

    def _post(self, w2, dtype) -> torch.Tensor:
        p = self.post
        if self.ssq is not None:  # the sum is in x already
            y, self.x = ops.post_norm(self.x, None, None, 1.0, p.w, w2, p.eps, dtype)
        else:
            y, self.x = ops.post_norm(self.x, self.delta, p.bias, p.alpha, p.w, w2, p.eps, dtype)
        self.delta = self.post = self.ssq = self.rows = None
        return y

    def last_norm(self, w, eps: float, offset: float, dtype) -> torch.Tensor:
        """The model's last norm on the finished stream."""
        if self.post is None:
            return self.norm(w, eps, offset, dtype)
        return self._post(w, dtype)


class CacheSlot:
    """What one mixer run keeps of the past: named tensors with the batch first. `per_token` names the
    tensors with one row per token and the dimension of the rows (at most `limit` of them, 0: one for
    every token; grown by `reserve`), the others are fixed-size state. `rope`: the mixer's rotary tables."""

    def __init__(self, max_len: int, device, rope=None, per_token: Optional[Dict[str, int]] = None, limit: int = 0,
                 **tensors):
        self.t = tensors
        self.rope, self.per_token, self.limit = rope, per_token or {}, limit
        self.device = device
        self.cos = self.sin = None
        self.grow(max_len)

    def grow(self, max_len: int):
        # the slot keeps its own reference to the rotary tables: a captured decode step reads them
        # by address, also after a longer cache made the shared RotaryCache extend
        if self.rope is not None:
            self.rope.ensure(max_len)
            self.cos, self.sin = self.rope.tables(self.device)

    def nbytes(self) -> int:
        return sum(v.numel() * v.element_size() for v in self.t.values())

    def keep_rows(self, rows: torch.Tensor) -> "CacheSlot":
        out = CacheSlot.__new__(CacheSlot)
        out.__dict__.update(self.__dict__)
        out.t = {k: v.index_select(0, rows.to(v.device)) for k, v in self.t.items()}
        return out

    def reserve(self, max_len: int):
        n = min(max_len, self.limit) if self.limit else max_len
        for name, dim in self.per_token.items():
            old = self.t[name]
            if n <= old.shape[dim]:
                continue
            shape = list(old.shape)
            shape[dim] = n
            new = torch.zeros(shape, dtype=old.dtype, device=old.device)
            new.narrow(dim, 0, old.shape[dim]).copy_(old)
            self.t[name] = new
        self.grow(max_len)


class LatentAttention(nn.Module):
    """Multi-head attention whose keys and values are projections of one cached latent per token
    (plus one rotated key part shared by the heads), inside a sliding window."""

    def __init__(self, cfg: ModelConfig, m: dict, device=None, dtype=None):
        super().__init__()
        H = cfg.hidden_size
        self.eps = cfg.norm_eps
        self.heads, self.dim, self.rot, self.vdim = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
        self.q_rank, self.kv_rank = m["q_rank"], m["kv_rank"]
        self.scale, self.window = float(m["scale"]), window(m)
        self.rope_key = (m["rot"]["dims"], float(m["rot"]["base"]))
        self.rope = None  # the model's shared RotaryCache of rope_key
        self.in_proj = _param(self.q_rank + self.kv_rank + self.rot, H, device=device, dtype=dtype)
        self.q_norm_w = _param(self.q_rank, device=device, dtype=dtype)
        self.kv_norm_w = _param(self.kv_rank, device=device, dtype=dtype)
        self.q_up = _param(self.heads * (self.dim + self.rot), self.q_rank, device=device, dtype=dtype)
        # [all heads' unrotated keys; all heads' values]
        self.kv_up = _param(self.heads * (self.dim + self.vdim), self.kv_rank, device=device, dtype=dtype)
        self.o_proj = _param(H, self.heads * self.vdim, device=device, dtype=dtype)

    def new_slot(self, batch: int, max_len: int, device, dtype) -> CacheSlot:
        return CacheSlot(max_len, device, self.rope, per_token={"latent": 1}, latent=torch.zeros(
            (batch, max_len, self.kv_rank + self.rot), device=device, dtype=dtype))

    def mix(self, down: torch.Tensor, cache, slot: CacheSlot, lin=ops.stream_linear) -> torch.Tensor:
        """down = in_proj output [B, T, q_rank + kv_rank + rot] -> heads' outputs [B, T, heads * vdim];
        the new tokens' latents go into the slot."""
        _, T, _ = down.shape
        latent = slot.t["latent"]
        cq = ops.latent.prepare(down, self.q_norm_w, self.kv_norm_w, self.eps, latent, cache.slot,
                                cache.kv_start, slot.cos, slot.sin, base=cache.len)
        q = lin(cq, self.q_up)
        if T == 1 and cache.len > 0:
            return ops.latent.decode(q, latent, self.kv_up, self.heads, self.dim, self.rot, self.vdim,
                                     self.scale, self.window, cache.slot, cache.kv_start, slot.cos,
                                     slot.sin, base=cache.len)
        # prefill (of a whole prompt, or a portion after earlier ones): keys and values of every
        # visible token are projected up once
        lo = max(0, cache.len + 1 - self.window) if self.window else 0
        seen = latent[:, lo:cache.len + T]
        kv = ops.stream_linear(seen[..., :self.kv_rank].contiguous(), self.kv_up)
        return ops.latent.prefill(q, kv, seen[..., self.kv_rank:], self.heads, self.dim, self.rot, self.vdim,
                                  self.scale, self.window, cache.kv_start, slot.cos, slot.sin,
                                  q_base=cache.len, k_base=lo)

    def forward(self, h, cache, slot):
        return ops.stream_linear(self.mix(ops.stream_linear(h, self.in_proj), cache, slot), self.o_proj)

    def matrices(self):
        return (self.in_proj, self.q_up, self.o_proj)


class Retention(nn.Module):
    """Linear attention with one fixed decay per head; its past is one fp32 state per head."""

    def __init__(self, cfg: ModelConfig, m: dict, device=None, dtype=None):
        super().__init__()
        H = cfg.hidden_size
        self.eps = cfg.norm_eps
        self.heads, self.dim, self.vdim = m["heads"], m["dim"], m["vdim"]
        self.rope_key = (m["rot"]["dims"], float(m["rot"]["base"]))
        self.rope = None
        self.decay = [float(x) for x in m["decay"]]
        self._decay = {}
        # rows [q; k; v; g]
        self.in_proj = _param(2 * self.heads * (self.dim + self.vdim), H, device=device, dtype=dtype)
        self.o_proj = _param(H, self.heads * self.vdim, device=device, dtype=dtype)

    def decays(self, device) -> torch.Tensor:
        """[2, heads] fp32: the decays and their base-2 logarithms."""
        t = self._decay.get(device)
        if t is None:
            d = torch.tensor(self.decay, dtype=torch.float64)
            t = torch.stack([d, d.log2().clamp(min=-1e4)]).float().to(device)
            self._decay[device] = t
        return t

    def new_slot(self, batch: int, max_len: int, device, dtype) -> CacheSlot:
        return CacheSlot(max_len, device, self.rope, state=torch.zeros(
            (batch, self.heads, self.vdim, self.dim), device=device, dtype=torch.float32))

    def mix(self, qkvg: torch.Tensor, cache, slot: CacheSlot, lin=None) -> torch.Tensor:
        _, T, _ = qkvg.shape
        args = (self.heads, self.dim, self.vdim, self.rope_key[0], self.eps, self.decays(qkvg.device),
                slot.t["state"], cache.slot, cache.kv_start, slot.cos, slot.sin)
        if T == 1 and cache.len > 0:
            return ops.retention.decode(qkvg, *args, base=cache.len)
        return ops.retention.prefill(qkvg, *args, base=cache.len)

    def forward(self, h, cache, slot):
        return ops.stream_linear(self.mix(ops.stream_linear(h, self.in_proj), cache, slot), self.o_proj)

    def matrices(self):
        return (self.in_proj, self.o_proj)


class GatedRecurrence(nn.Module):
    """Griffin's recurrent block: a gelu branch times a real-gated linear recurrence behind a short
    convolution; its past is one fp32 state per channel and the convolution's last inputs."""

    rope_key = None

    def __init__(self, cfg: ModelConfig, m: dict, device=None, dtype=None):
        super().__init__()
        H, W, nb = cfg.hidden_size, m["width"], m["blocks"]
        self.width, self.taps = W, m["conv"]
        self.in_proj = _param(2 * W, H, device=device, dtype=dtype)  # rows [y; x]
        self.in_bias = _param(2 * W, device=device, dtype=dtype)
        self.conv_w = _param(W, self.taps, device=device, dtype=dtype)
        self.conv_b = _param(W, device=device, dtype=dtype)
        self.gates = _param(2 * nb, W // nb, W // nb, device=device, dtype=dtype)  # blocks of r, then of i
        self.gates_b = _param(2 * nb, W // nb, device=device, dtype=dtype)
        self.lam = _param(W, device=device, dtype=dtype)
        self.o_proj = _param(H, W, device=device, dtype=dtype)
        self.o_bias = None

    def new_slot(self, batch: int, max_len: int, device, dtype) -> CacheSlot:
        return CacheSlot(max_len, device, state=torch.zeros((batch, self.width), device=device, dtype=torch.float32),
                         hist=torch.zeros((batch, self.taps, self.width), device=device, dtype=dtype))

    def mix(self, yx: torch.Tensor, cache, slot: CacheSlot) -> torch.Tensor:
        run = ops.lru.decode if yx.shape[1] == 1 and cache.len > 0 else ops.lru.prefill
        return run(yx, self.in_bias, self.conv_w, self.conv_b, self.gates, self.gates_b, self.lam, slot.t["state"],
                   slot.t["hist"], cache.slot, cache.kv_start, base=cache.len)

    def matrices(self):
        return (self.in_proj, self.o_proj)


class GatedLinearAttention(nn.Module):
    """Linear attention with a decay per key channel and token; its past is one fp32 state per head."""

    rope_key = None

    def __init__(self, cfg: ModelConfig, m: dict, device=None, dtype=None):
        super().__init__()
        H = cfg.hidden_size
        self.eps, self.tau = cfg.norm_eps, float(m["tau"])
        self.heads, self.dim, self.vdim = m["heads"], m["dim"], m["vdim"]
        # rows [q; k; v; g; first decay projection]
        self.in_proj = _param(2 * self.heads * (self.dim + self.vdim) + decay_rank(m), H, device=device, dtype=dtype)
        self.decay_proj = _param(self.heads * self.dim, decay_rank(m), device=device, dtype=dtype)
        self.decay_b = _param(self.heads * self.dim, device=device, dtype=dtype)
        self.norm_w = _param(self.vdim, device=device, dtype=dtype)
        self.o_proj = _param(H, self.heads * self.vdim, device=device, dtype=dtype)
        self.o_bias = None

    def new_slot(self, batch: int, max_len: int, device, dtype) -> CacheSlot:
        return CacheSlot(max_len, device, state=torch.zeros((batch, self.heads, self.vdim, self.dim), device=device,
                                                            dtype=torch.float32))

    def mix(self, proj: torch.Tensor, cache, slot: CacheSlot) -> torch.Tensor:
        run = ops.gla.decode if proj.shape[1] == 1 and cache.len > 0 else ops.gla.prefill
        return run(proj, self.decay_proj, self.decay_b, self.norm_w, self.heads, self.dim, self.vdim, self.tau, self.eps,
                   slot.t["state"], cache.slot, cache.kv_start, base=cache.len)

    def matrices(self):
        return (self.in_proj, self.o_proj)


class ChunkAttention(nn.Module):
    """Grouped-query attention inside chunks of the sequence, query and key normed over their whole
    projections, the values being the projected keys; its past is the keys and values of one chunk."""

    def __init__(self, cfg: ModelConfig, m: dict, device=None, dtype=None):
        super().__init__()
        H, n, g, d = cfg.hidden_size, m["heads"], m["kv_heads"], m["dim"]
        self.rope_key = (m["rot"]["dims"], float(m["rot"]["base"]))
        self.rope = None
        self.h = ops.chunk_attention.Heads(n, g, d, m["vdim"], m["rot"]["dims"], n * d, window(m), float(m["scale"]),
                                           cfg.norm_eps)
        self.in_proj = _param((n + g) * d, H, device=device, dtype=dtype)  # rows [q; k]
        self.in_bias = _param((n + g) * d, device=device, dtype=dtype)
        self.q_norm_w = _param(n * d, device=device, dtype=dtype)
        self.k_norm_w = _param(g * d, device=device, dtype=dtype)
        self.o_proj = _param(H, n * m["vdim"], device=device, dtype=dtype)
        self.o_bias = _param(H, device=device, dtype=dtype)

    def new_slot(self, batch: int, max_len: int, device, dtype) -> CacheSlot:
        h, rows = self.h, min(max_len, self.h.chunk) if self.h.chunk else max_len
        return CacheSlot(max_len, device, self.rope, per_token={"k": 2, "v": 2}, limit=h.chunk,
                         k=torch.zeros((batch, h.kv_heads, rows, h.dim), device=device, dtype=dtype),
                         v=torch.zeros((batch, h.kv_heads, rows, h.vdim), device=device, dtype=dtype))

    def mix(self, qk: torch.Tensor, cache, slot: CacheSlot) -> torch.Tensor:
        att, kc, vc = ops.chunk_attention, slot.t["k"], slot.t["v"]
        w = (self.in_bias, self.q_norm_w, self.k_norm_w)
        if qk.shape[1] == 1 and cache.len > 0:
            return att.decode(qk, *w, kc, vc, self.h, cache.slot, cache.kv_start, slot.cos, slot.sin, base=cache.len)
        q, k, v = att.prepare(qk, *w, self.h, cache.kv_start, slot.cos, slot.sin, base=cache.len)
        o = att.prefill(q, k, v, kc, vc, self.h, cache.kv_start, base=cache.len)
        att.store(k, v, kc, vc, self.h, cache.kv_start, base=cache.len)
        return o

    def matrices(self):
        return (self.in_proj, self.o_proj)


MIXERS = {"latent_attention": LatentAttention, "retention": Retention, "rglru": GatedRecurrence,
          "gla": GatedLinearAttention, "attention": ChunkAttention}


class TokenSide(nn.Module):
    """Per-layer token input: a gated slice of a second embedding, projected up and RMS-normed."""

    def __init__(self, cfg: ModelConfig, device=None, dtype=None):
        super().__init__()
        self.gate = _param(cfg.token_side_dim, cfg.hidden_size, device=device, dtype=dtype)
        self.proj = _param(cfg.hidden_size, cfg.token_side_dim, device=device, dtype=dtype)
        self.norm_w = _param(cfg.hidden_size, device=device, dtype=dtype)


class StreamLayer(nn.Module):
    """One layer of a per-layer design: norm, mixer, [norm, feed-forward], [per-layer token input]."""

    def __init__(self, cfg: ModelConfig, index: int, device=None, dtype=None):
        super().__init__()
        from .transformer import MLP

        spec = cfg.layer_specs[index]
        self.cfg, self.index = cfg, index
        H = cfg.hidden_size
        self.ln1_w = _param(H, device=device, dtype=dtype)
        self.mix = MIXERS[spec["type"]](cfg, spec["mixer"], device, dtype)
        self.mlp = None
        if spec.get("mlp"):
            self.ln2_w = _param(H, device=device, dtype=dtype)
            self.mlp = MLP(dataclasses.replace(cfg, intermediate_size=spec["mlp"]["ff"]), device, dtype)
        self.side = TokenSide(cfg, device, dtype) if cfg.token_side_dim else None
        self.recompute = None

    def fused_ok(self, rows: int) -> bool:
        """A decode step of this layer can run on the fused projections (norm in front, stream add /
        activation / gate behind)."""
        ws = self.mix.matrices()
        if self.mlp is not None:
            ws += (self.mlp.up_proj, self.mlp.down_proj)
        if self.side is not None:
            ws += (self.side.gate, self.side.proj)
        return ops.stream.fused_ok(rows, self.ln1_w.dtype, *ws)

    def decode_fused(self, s: Stream, ids: torch.Tensor, side_embed, cache, slot: CacheSlot) -> Stream:
        cfg, st = self.cfg, ops.stream
        eps, off = cfg.norm_eps, cfg.norm_offset
        h = s.norm(self.ln1_w, eps, off, self.ln1_w.dtype)
        a = self.mix.mix(st.fused_linear(h, self.mix.in_proj), cache, slot, st.fused_linear)
        # each add hands the next reader of x its rows: weighted for a norm, plain for the side gate
        h, ssq = st.fused_add(a, self.mix.o_proj, s.x, self.ln2_w if self.mlp is not None else None, off)
        if self.mlp is not None:
            m = st.fused_linear(h, self.mlp.up_proj, ssq, eps, relu2=True)
            h, _ = st.fused_add(m, self.mlp.down_proj, s.x, None, 0.0)
        if self.side is not None:
            g = st.fused_gate(h, self.side.gate, ids, side_embed, self.index * cfg.token_side_dim)
            s.delta, s.delta_w = st.fused_linear(g, self.side.proj), self.side.norm_w
        return s

    def forward(self, s: Stream, ids: torch.Tensor, side_embed, cache, slot: CacheSlot) -> Stream:
        cfg, dt = self.cfg, self.ln1_w.dtype
        if ids.shape[1] == 1 and not torch.is_grad_enabled() and self.fused_ok(ids.shape[0]):
            return self.decode_fused(s, ids, side_embed, cache, slot)
        h = s.norm(self.ln1_w, cfg.norm_eps, cfg.norm_offset, dt)
        s.delta = self.mix(h, cache, slot)
        if self.mlp is not None:
            h = s.norm(self.ln2_w, cfg.norm_eps, cfg.norm_offset, dt)
            s.delta = self.mlp(h)
        if self.side is not None:
            side = self.side
            g = ops.side_gate(ops.stream_linear(s.cast(cfg.norm_eps, dt), side.gate), ids, side_embed,
                              self.index * cfg.token_side_dim)
            s.delta, s.delta_w = ops.stream_linear(g, side.proj), side.norm_w
        return s


class PostNormLayer(nn.Module):
    """One layer with its norms after the sums: x <- norm(alpha x + mixer(x)), [x <- norm(alpha x + ff(x))]."""

    def __init__(self, cfg: ModelConfig, index: int, device=None, dtype=None):
        super().__init__()
        from .transformer import MLP

        spec = cfg.layer_specs[index]
        self.cfg, self.index = cfg, index
        H = cfg.hidden_size
        self.ln1_w = _param(H, device=device, dtype=dtype)
        self.mix = MIXERS[spec["type"]](cfg, spec["mixer"], device, dtype)
        self.mlp = None
        if spec.get("mlp"):
            self.ln2_w = _param(H, device=device, dtype=dtype)
            self.mlp = MLP(dataclasses.replace(cfg, intermediate_size=spec["mlp"]["ff"]), device, dtype)
        self.recompute = None

    def fused_ok(self, rows: int) -> bool:
        """A decode step of this layer can run on the fused projections (norm in front, sum and norm /
        gated unit behind)."""
        ws = self.mix.matrices()
        if self.mlp is not None:
            ws += (self.mlp.up_proj, self.mlp.down_proj)
        return ops.stream.fused_ok(rows, self.ln1_w.dtype, *ws)

    def decode_fused(self, s: Stream, cache, slot: CacheSlot) -> Stream:
        cfg, st = self.cfg, ops.stream
        eps, alpha = cfg.norm_eps, cfg.postln_alpha
        if s.ssq is None:
            h, prev = s.cast(eps, self.ln1_w.dtype), (None, None)
        else:
            h, prev = s.rows, (s.ssq, s.post.w)
        a = self.mix.mix(st.fused_linear(h, self.mix.in_proj, prev[0], eps), cache, slot)
        w = self.ln1_w
        h, ssq = st.fused_post(a, self.mix.o_proj, s.x, alpha, self.mix.o_bias, *prev, w, eps)
        if self.mlp is not None:
            m = st.fused_geglu(h, self.mlp.up_proj, ssq, eps)
            h, ssq = st.fused_post(m, self.mlp.down_proj, s.x, alpha, None, ssq, w, self.ln2_w, eps)
            w = self.ln2_w
        s.rows, s.ssq, s.post = h, ssq, PostNorm(w, alpha, eps)
        return s

    def forward(self, s: Stream, ids: torch.Tensor, side_embed, cache, slot: CacheSlot) -> Stream:
        cfg, dt = self.cfg, self.ln1_w.dtype
        if ids.shape[1] == 1 and not torch.is_grad_enabled() and self.fused_ok(ids.shape[0]):
            return self.decode_fused(s, cache, slot)
        a = self.mix.mix(ops.stream_linear(s.cast(cfg.norm_eps, dt), self.mix.in_proj), cache, slot)
        s.delta = ops.stream_linear(a, self.mix.o_proj)
        s.post = PostNorm(self.ln1_w, cfg.postln_alpha, cfg.norm_eps, self.mix.o_bias)
        if self.mlp is not None:
            s.delta = self.mlp(s.cast(cfg.norm_eps, dt))
            s.post = PostNorm(self.ln2_w, cfg.postln_alpha, cfg.norm_eps)
        return s


def build_layers(cfg: ModelConfig, device=None, dtype=None) -> List[nn.Module]:
    """The layers of a per-layer design; mixers with equal rotary settings share one table."""
    kind = StreamLayer if cfg.postln_alpha is None else PostNormLayer
    layers = [kind(cfg, i, device, dtype) for i in range(cfg.num_layers)]
    ropes = {}
    for layer in layers:
        key = layer.mix.rope_key
        if key is None:
            continue
        if key not in ropes:
            ropes[key] = ops.RotaryCache(key[0], key[1], 256)
        layer.mix.rope = ropes[key]
    return layers
