"""Zenevik through the framework (config, loading, caches, generation, trace runner) and its ops,
against the plain float64 oracle of zenevik_oracle.py. Every test runs on the CPU forms of the ops
and, in the GPU tier, on the HIP kernels in fp32 and bf16."""
import json
import os
import subprocess
import sys

import pytest
import torch

import zenevik_oracle as O
from distributed_llm_alignment_amd import ops
from distributed_llm_alignment_amd.eval.trace_run import TraceRunner
from distributed_llm_alignment_amd.models import build_model, generate, get_config, load_causal_lm, save_hf_pretrained
from distributed_llm_alignment_amd.models.config import ModelConfig
from distributed_llm_alignment_amd.ops.chunk_attention import Heads
from test_vufilorn import FP32, GPU, ROOT, WHERE, close, new_cache, rel, rnd, run, tokens_of

CONFIGS = {
    # every mixer, with and without a feed-forward, sizes that are multiples of 8
    "mix": O.config(72, 96, [(O.lru(96, 4, 3), None), (O.gated(3, 16, 24, 8.0, 8), 88), (O.attn(4, 2, 24, 16, 11, 0.3), None),
                             (O.lru(64, 1, 4), 40), (O.attn(3, 3, 16, 16, 7, 0.4, 500.0), 64)]),
    # nothing a multiple of anything; one block per channel; rotation of a few dimensions
    "odd": O.config(50, 67, [(O.lru(35, 5, 2), 35), (O.gated(3, 10, 7, 3.0, 5), None), (O.attn(5, 5, 9, 6, 5, 0.5), 30),
                             (O.lru(21, 21, 6), None), (O.gated(4, 11, 13, 2.0, 3), 31)], alpha=2.5, cap=7.0, eps=1e-2),
    # one head, chunks of one token (a token sees itself only), a convolution of one tap
    "min": O.config(32, 40, [(O.lru(16, 1, 1), None), (O.attn(1, 1, 8, 2, 1, 1.0), 16), (O.gated(1, 8, 16, 16.0, 1), None)]),
    # head and block sizes of the large models' kernels; decays of very different speeds
    "wide": O.config(128, 64, [(O.lru(512, 2, 4), 96), (O.gated(2, 128, 256, 16.0, 16), 64), (O.attn(4, 1, 128, 64, 70, 0.09), None),
                               (O.gated(1, 256, 64, 0.25, 40), None), (O.attn(1, 1, 256, 256, 100, 0.06), 64)]),
    # 20 query heads on one key head (two groups of 16 in decode), blocks of more than 128 channels
    "heads": O.config(256, 128, [(O.lru(320, 2, 5), 256), (O.attn(20, 1, 32, 32, 48, 0.2), 512), (O.gated(4, 64, 64, 2.0, 16), 512)],
                      alpha=3.0),
}
_CACHE = {}


def model_of(name, where):
    """(config, weights, framework model) of CONFIGS[name], built once per place and dtype."""
    dev, dt = where
    key = (name, dev, dt)
    if key not in _CACHE:
        cfg = CONFIGS[name]
        P = O.weights(cfg, seed=sum(map(ord, name)))
        m = build_model(ModelConfig.from_hf(cfg), device=dev, dtype=dt, init=False)
        m.load_hf_state_dict(P, strict=True)
        _CACHE[key] = (cfg, P, m.eval())
    return _CACHE[key]


def want_of(cfg, P, toks):
    key = (id(P), tuple(toks))
    if key not in _CACHE:
        _CACHE[key] = O.forward(toks, P, cfg)
    return _CACHE[key]


# ----------------------------------------------------------------------------------- whole models
@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("name", list(CONFIGS))
@torch.no_grad()
def test_prompt_matches_oracle(name, where):
    cfg, P, m = model_of(name, where)
    for n in (1, 2, 37, 150):
        toks = tokens_of(cfg, n)
        got = m.logits(m(torch.tensor([toks], device=where[0])))[0]
        assert got.dtype == torch.float32 and got.abs().max() <= cfg["logit_softcap"]
        close(got, want_of(cfg, P, toks), where)


@pytest.mark.parametrize("where", FP32)
@pytest.mark.parametrize("name", ["mix", "odd"])
@torch.no_grad()
def test_stream_after_every_layer(name, where):
    cfg, P, m = model_of(name, where)
    toks, want, got = tokens_of(cfg, 41, 3), [], []
    O.forward(toks, P, cfg, want)

    def keep(_mod, _args, s):
        x = s.x.clone()
        y = ops.post_norm(x, s.delta, s.post.bias, s.post.alpha, s.post.w, None, s.post.eps, x.dtype)[1]
        got.append(y[0])

    hooks = [layer.register_forward_hook(keep) for layer in m.layers]
    m(torch.tensor([toks], device=where[0]))
    for h in hooks:
        h.remove()
    assert len(got) == len(want)
    for g, w in zip(got, want):
        rel(g, w, where, 2e-5)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("name", list(CONFIGS))
@torch.no_grad()
def test_token_by_token_matches_prompt(name, where):
    """Decoding from the first token on, past every chunk."""
    cfg, P, m = model_of(name, where)
    toks = tokens_of(cfg, 110, 1)
    want = want_of(cfg, P, toks)
    cache = new_cache(m, 1, len(toks))
    got = torch.cat([run(m, [[t]], cache, where[0])[0] for t in toks])
    close(got, want, where)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("name", ["mix", "odd", "wide", "heads"])
@torch.no_grad()
def test_portions(name, where):
    """A prompt cut into portions of several sizes, down to two tokens and mixed with single ones:
    portions that start, end and lie across chunk borders, and shorter than the convolution."""
    cfg, P, m = model_of(name, where)
    toks = tokens_of(cfg, 150, 2)
    want = want_of(cfg, P, toks)
    for cuts in ([2] * 75, [100, 50], [64, 64, 22], [1, 2, 3, 5, 16, 17, 32, 33, 41], [149, 1], [70, 70, 10], [69, 2, 68, 11]):
        cache, at, got = new_cache(m, 1, len(toks)), 0, []
        for c in cuts:
            got.append(run(m, [toks[at:at + c]], cache, where[0])[0])
            at += c
        assert at == len(toks)
        close(torch.cat(got), want, where)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("name", ["mix", "odd", "wide", "heads"])
@torch.no_grad()
def test_unequal_batch_against_alone(name, where):
    """Left-padded rows of very different lengths, in two portions, then decoded together; rows leave
    half-way. Rows that are still padding in the first portion start in the second."""
    cfg, P, m = model_of(name, where)
    lens, steps, cut = [1, 130, 2, 67, 12], 24, 75
    seqs = [tokens_of(cfg, n + steps, 3 + i) for i, n in enumerate(lens)]
    T = max(lens)
    rows = [[0] * (T - n) + s[:n] for n, s in zip(lens, seqs)]
    for parts in ([T], [cut, T - cut]):
        cache, at, got = new_cache(m, len(lens), T + steps, [T - n for n in lens]), 0, []
        for c in parts:
            got.append(run(m, [r[at:at + c] for r in rows], cache, where[0]))
            at += c
        got = torch.cat(got, 1)
        out = {i: [got[i, T - n:]] for i, n in enumerate(lens)}
        alive = list(range(len(lens)))
        for t in range(steps):
            if t == 10:  # rows 1 and 2 end; the others keep what they hold
                cache = cache.keep_rows([alive.index(i) for i in (4, 0, 3)])
                alive = [4, 0, 3]
            got = run(m, [[seqs[i][lens[i] + t]] for i in alive], cache, where[0])
            for r, i in enumerate(alive):
                out[i].append(got[r])
        for i, s in enumerate(seqs):
            lg = torch.cat(out[i])
            close(lg, want_of(cfg, P, s)[:lg.shape[0]], where)


@pytest.mark.parametrize("where", FP32)
@torch.no_grad()
def test_cache_reused_and_grown(where):
    """A cache that is reset keeps nothing of the last batch; one that grows keeps everything; the
    attention cache never holds more than one chunk."""
    cfg, P, m = model_of("mix", where)
    a, b = tokens_of(cfg, 60, 9), tokens_of(cfg, 60, 10)
    cache = new_cache(m, 1, 60, [0])
    for toks in (a, b):
        cache.reset(torch.zeros(1, dtype=torch.int32, device=where[0]))
        got = torch.cat([run(m, [toks[:40]], cache, where[0])[0]] + [run(m, [[t]], cache, where[0])[0] for t in toks[40:]])
        close(got, want_of(cfg, P, toks), where)
    assert cache.slots[2].t["k"].shape[2] == 11 and cache.slots[4].t["v"].shape[2] == 7
    small = new_cache(m, 1, 5)
    assert small.slots[2].t["k"].shape[2] == 5
    got = torch.cat([run(m, [a[:5]], small, where[0])[0]] + [run(m, [[t]], small, where[0])[0] for t in a[5:]])
    close(got, want_of(cfg, P, a), where)
    assert small.slots[2].t["k"].shape[2] == 11


@pytest.mark.parametrize("where", WHERE)
@torch.no_grad()
def test_long_decoding(where):
    cfg, P, m = model_of("mix", where)
    toks = tokens_of(cfg, 400, 11)
    cache = new_cache(m, 1, len(toks))
    got = torch.cat([run(m, [toks[:5]], cache, where[0])[0]] + [run(m, [[t]], cache, where[0])[0] for t in toks[5:]])
    close(got, want_of(cfg, P, toks), where)


def _plant(cfg, P, what):
    """The oracle with one mistake in it."""
    c, Q = json.loads(json.dumps(cfg)), dict(P)
    if what == "chunk":
        c["layers"][2]["mixer"]["mask"]["size"] += 1
    elif what == "tau":
        c["layers"][1]["mixer"]["tau"] *= 1.02
    elif what == "alpha":
        c["postln_alpha"] *= 1.01
    elif what == "softcap":
        c["logit_softcap"] *= 1.05
    elif what == "tap order":
        Q["l0.mix.conv"] = P["l0.mix.conv"].flip(1)
    elif what == "gates swapped":
        Q["l3.mix.ra"], Q["l3.mix.ri"] = P["l3.mix.ri"], P["l3.mix.ra"]
    elif what == "key bias":
        Q["l2.mix.k.b"] = P["l2.mix.k.b"] * 0.98
    elif what == "rotary base":
        c["layers"][2]["mixer"]["rot"]["base"] *= 1.1
    elif what == "output bias":
        Q["l2.mix.o.b"] = P["l2.mix.o.b"] * 0.95
    return O.forward(tokens_of(cfg, 37), Q, c)


@pytest.mark.parametrize("what", ["chunk", "tau", "alpha", "softcap", "tap order", "gates swapped", "key bias", "rotary base",
                                  "output bias"])
@torch.no_grad()
def test_tolerance_sees_planted_mistakes(what):
    cfg, P, m = model_of("mix", ("cpu", torch.float32))
    got = m.logits(m(torch.tensor([tokens_of(cfg, 37)])))[0]
    with pytest.raises(AssertionError):
        close(got, _plant(cfg, P, what), ("cpu", torch.float32), f32=1e-3)


# ------------------------------------------------------------------------------- mechanisms alone
def f64(t):
    return t.double().cpu()


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("H", [48, 50, 1000, 2048, 5000])
def test_post_norm(H, where):
    x = torch.randn(3, 5, H, generator=torch.Generator().manual_seed(H)).to(where[0]) * 3
    d, b, w, w2 = rnd(where, 3, 5, H), rnd(where, H, seed=3), rnd(where, H, seed=1), rnd(where, H, seed=2)
    for delta, bias, last in ((d, None, None), (d, b, None), (d, b, w2), (None, None, w2)):
        s = 1.7 * f64(x) + (0 if delta is None else f64(d)) + (0 if bias is None else f64(b))
        want = O.rms(s, 1e-3) * f64(w)
        y, xn = ops.post_norm(x.clone(), delta, bias, 1.7, w, last, 1e-3, where[1])
        assert xn.dtype == torch.float32 and y.dtype == where[1]
        rel(xn, want, where, 2e-6, 2e-6)  # the stream is fp32 in both modes
        rel(y, want if last is None else O.rms(want, 1e-3) * f64(w2), where)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("F", [40, 37])
def test_geglu_softcap(F, where):
    u = rnd(where, 2, 3, 2 * F, scale=2.0)
    want = O.gelu_tanh(f64(u)[..., :F]) * f64(u)[..., F:]
    rel(ops.geglu(u), want, where)
    z = rnd(where, 3, 4, F, scale=9.0)
    got = ops.softcap(z, 5.0)
    assert got.dtype == torch.float32
    rel(got, O.softcap(f64(z), 5.0), where, 2e-6, 2e-6)


@GPU
@pytest.mark.parametrize("M", [1, 5, 16, 17, 32])
@pytest.mark.parametrize("N,K", [(50, 72), (256, 2048), (2048, 1024), (33, 264)])
def test_fused_decode_projections(M, N, K):
    """Sum and norm behind a projection (with and without a norm pending on x), the gated unit and the
    soft cap, against float64."""
    where = ("cuda", torch.bfloat16)
    a, w, st = rnd(where, M, 1, K), rnd(where, N, K, scale=K ** -0.5), ops.stream
    want = f64(a)[:, 0] @ f64(w).T
    x, nw, rw, bias = torch.randn(M, 1, N, device="cuda") * 2, rnd(where, N), rnd(where, N, seed=1), rnd(where, N, seed=2)
    ssq = torch.stack([p.pow(2).sum(-1) for p in x[:, 0].split(16, -1)], -1).contiguous()
    for res, rwt, b in ((None, None, None), (ssq, rw, None), (ssq, rw, bias)):
        xi = x.clone()
        h, sq = st.fused_post(a, w, xi, 1.6, b, res, rwt, nw, 1e-3)
        prev = f64(x)[:, 0] if res is None else O.rms(f64(x)[:, 0], 1e-3) * f64(rw)
        xw = 1.6 * prev + want + (0 if b is None else f64(b))
        rel(xi[:, 0], xw, where, b16=2e-5)  # the stream is fp32
        rel(sq.sum(1), (xw ** 2).sum(1), where, b16=2e-5)
        rel(h[:, 0], xw * f64(nw), where)
    u = rnd(where, 2 * N, K, seed=4, scale=K ** -0.5)
    scale = 1 / torch.sqrt(f64(ssq).sum(1, keepdim=True) / K + 1e-3)
    gu = f64(a)[:, 0] @ f64(u).T
    rel(st.fused_geglu(a, u)[:, 0], O.gelu_tanh(gu[:, :N]) * gu[:, N:], where)
    gu = gu * scale
    rel(st.fused_geglu(a, u, ssq, 1e-3)[:, 0], O.gelu_tanh(gu[:, :N]) * gu[:, N:], where)
    got = ops.head_logits(a * 4, w, 3.0)
    assert got.dtype == torch.float32
    rel(got[:, 0], O.softcap(4 * want, 3.0), where)


def _lru_case(where, W, nb, taps, seed=0):
    P = O.weights(O.config(8, 4, [(O.lru(W, nb, taps), None)]), seed=seed + W)
    t = {k.split("mix.")[1]: v.to(where[0], where[1]) for k, v in P.items() if ".mix." in k}
    args = (torch.cat([t["y.b"], t["x.b"]]), t["conv"], t["conv.b"], torch.cat([t["ra"], t["ri"]]), torch.cat([t["ra.b"], t["ri.b"]]),
            t["lam"])
    return {k: f64(v) for k, v in t.items()}, args


def _lru_oracle(yx, t, W, u_dtype):
    """One row's outputs and final state; u rounded as the kernels round it."""
    y, x = O.gelu_tanh(f64(yx)[:, :W] + t["y.b"]), f64(yx)[:, W:] + t["x.b"]
    u = f64(O.causal_conv(x, t["conv"], t["conv.b"]).to(u_dtype))
    S = O.lru_scan(u, O.block_gate(u, t["ra"], t["ra.b"]), O.block_gate(u, t["ri"], t["ri.b"]), t["lam"])
    return S * y, S[-1]


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("W,nb,taps", [(64, 4, 4), (35, 5, 3), (7, 7, 1), (320, 2, 6), (512, 2, 4), (200, 1, 2), (312, 1, 3)])
def test_lru_alone(W, nb, taps, where):
    """Tiles and chunks of tokens, a second portion, one shorter than the convolution, decode; a padded
    row whose padding holds NaN, and stale state and history that a fresh sequence must not see."""
    t, args = _lru_case(where, W, nb, taps)
    T1, T2, T3, steps, start = 301, 70, 2, 9, 37
    T = T1 + T2 + T3 + steps
    x = rnd(where, 2, T, 2 * W, seed=5, scale=1.5)
    if where[0] == "cuda":
        x[1, :start] = float("nan")
    state = torch.full((2, W), 1e6, device=where[0])
    hist = torch.full((2, taps, W), 300.0, device=where[0], dtype=where[1])
    kv0 = torch.tensor([0, start], dtype=torch.int32, device=where[0])
    slot, got, at = torch.zeros(1, dtype=torch.long, device=where[0]), [], 0
    for n in [T1, T2, T3] + [1] * steps:
        slot.fill_(at)
        op = ops.lru.decode if n == 1 else ops.lru.prefill
        got.append(op(x[:, at:at + n].contiguous(), *args, state, hist, slot, kv0, base=at))
        at += n
    got = torch.cat(got, 1)
    for b, s in ((0, 0), (1, start)):
        want, S = _lru_oracle(x[b, s:], t, W, where[1])
        rel(got[b, s:], want, where, 3e-5)
        rel(state[b], S, where, 1e-5, 2e-3)


@pytest.mark.parametrize("where", WHERE)
def test_lru_remembers_and_forgets(where):
    """Decays next to one and next to zero: sqrt(1 - a^2) keeps its digits, a far input stays."""
    W, nb = 16, 2
    t, args = _lru_case(where, W, nb, 1)
    lam = torch.linspace(-12, 6, W)
    args = (*args[:-1], lam.to(where[0], where[1]))
    t["lam"] = f64(args[-1])
    x = torch.zeros(1, 900, 2 * W)
    x[:, :, :W] = 1.0
    x[:, 3, W:] = 40.0  # one input far away from everything after it
    x = x.to(where[0], where[1])
    state, hist = torch.zeros(1, W, device=where[0]), torch.zeros(1, 1, W, device=where[0], dtype=where[1])
    got = ops.lru.prefill(x, *args, state, hist, torch.zeros(1, dtype=torch.long, device=where[0]), None, base=0)
    want, S = _lru_oracle(x[0], t, W, where[1])
    d = (f64(state)[0] - S).abs() / (S.abs() + 1e-3 * S.abs().max())
    assert d.max() < (3e-5 if where[1] == torch.float32 else 5e-3), d
    rel(got[0], want, where, 3e-5)


def _gla_case(where, H, d, vd, rank, T, tau, seed=0):
    proj = rnd(where, 2, T, 2 * H * (d + vd) + rank, seed=seed)
    a2, b, w = rnd(where, H * d, rank, seed=1, scale=1.5 * rank ** -0.5), rnd(where, H * d, seed=2, scale=2.0), rnd(where, vd, seed=3)
    return proj, a2, b, w


def _gla_oracle(proj, a2, b, w, H, d, vd, tau, eps):
    x = f64(proj)
    T, k = x.shape[0], H * d
    z = x[:, 2 * (k + H * vd):] @ f64(a2).T + f64(b)
    o, S = O.gla_recurrence(x[:, :k].view(T, H, d) * d ** -0.5, x[:, k:2 * k].view(T, H, d), x[:, 2 * k:2 * k + H * vd].view(T, H, vd),
                            O.log_sigmoid(z).view(T, H, d) / tau)
    g = x[:, 2 * k + H * vd:2 * (k + H * vd)]
    return (O.rms(o, eps) * f64(w)).reshape(T, H * vd) * O.silu(g), S


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("tau", [16.0, 1.0, 0.02])
@pytest.mark.parametrize("H,d,vd,rank", [(2, 16, 24, 16), (1, 10, 7, 3), (3, 128, 128, 16), (2, 64, 96, 8), (1, 256, 256, 40),
                                         (1, 40, 264, 8)])
def test_gla_alone(H, d, vd, rank, tau, where):
    """Chunked prefill, a second portion, decode, padding rows; NaN in padding must not spread, a stale
    state must not be seen. tau from slow decays to ones that forget within a token."""
    T1, T2, steps, start = 301, 70, 3, 37
    T = T1 + T2 + steps
    proj, a2, b, w = _gla_case(where, H, d, vd, rank, T, tau)
    state = torch.full((2, H, vd, d), 1e6, device=where[0])
    kv0 = torch.tensor([0, start], dtype=torch.int32, device=where[0])
    if where[0] == "cuda":
        proj[1, :start] = float("nan")
    slot, got, at = torch.zeros(1, dtype=torch.long, device=where[0]), [], 0
    for n in [T1, T2] + [1] * steps:
        slot.fill_(at)
        op = ops.gla.decode if n == 1 else ops.gla.prefill
        got.append(op(proj[:, at:at + n].contiguous(), a2, b, w, H, d, vd, tau, 1e-5, state, slot, kv0, base=at))
        at += n
    got = torch.cat(got, 1)
    for r, s in ((0, 0), (1, start)):
        want, S = _gla_oracle(proj[r, s:], a2, b, w, H, d, vd, tau, 1e-5)
        rel(got[r, s:], want, where, 5e-5)
        rel(state[r].transpose(1, 2), S, where, 2e-5, 1e-4)  # the state is fp32 in both modes


@pytest.mark.parametrize("where", WHERE)
def test_gla_far_key(where):
    """Slow decays and one large key far back: what is left of it stands out, across many chunks."""
    H, d, vd, T, tau = 2, 32, 32, 700, 64.0
    proj, a2, b, w = _gla_case(where, H, d, vd, 8, T, tau, seed=7)
    b = b + 6.0
    x = proj.clone()
    x[:, :, H * d:2 * H * d] *= 0.02
    x[:, 5, H * d:2 * H * d] *= 2000.0
    state = torch.zeros(2, H, vd, d, device=where[0])
    got = ops.gla.prefill(x, a2, b, w, H, d, vd, tau, 0.1, state, torch.zeros(1, dtype=torch.long, device=where[0]), None, base=0)
    want, _ = _gla_oracle(x[0], a2, b, w, H, d, vd, tau, 0.1)
    rel(got[0], want, where, 3e-4)  # (where q meets the far key at a right angle the norm amplifies)
    y = x[0].clone()
    y[5, H * d:2 * H * d] = 0
    without, _ = _gla_oracle(y, a2, b, w, H, d, vd, tau, 0.1)
    assert (without[-1] - want[-1]).abs().max() > 0.1 * want[-1].abs().max()  # it does stand out


def _attn_case(where, H, G, d, rot, B, T, chunk, scale, seed=0):
    row = rnd(where, B, T, (H + G) * d, seed=seed)
    w = (rnd(where, (H + G) * d, seed=1, scale=0.5), rnd(where, H * d, seed=2) + 1, rnd(where, G * d, seed=3) + 1)
    cos, sin = ops.RotaryCache(rot, 1000.0, T).tables(torch.device(where[0]))
    return row, w, Heads(H, G, d, d, rot, H * d, chunk, scale, 1e-4), cos, sin


def _attn_oracle(row, w, h):
    x = f64(row) + f64(w[0])
    T, nq = x.shape[0], h.heads * h.dim
    q = O.rotate((O.rms(x[:, :nq], h.eps) * f64(w[1])).view(T, h.heads, h.dim), 1000.0, h.rot)
    k = O.rotate((O.rms(x[:, nq:], h.eps) * f64(w[2])).view(T, h.kv_heads, h.dim), 1000.0, h.rot)
    return O.attend(q, k, x[:, nq:].view(T, h.kv_heads, h.dim), h.scale, h.chunk).reshape(T, -1)


def _attn_run(where, row, w, h, cos, sin, kv0, parts):
    """The portions `parts` of the rows (1: a decode step), through a cache full of stale values."""
    B, T = row.shape[:2]
    rows = min(T, h.chunk) if h.chunk else T
    kc = torch.full((B, h.kv_heads, rows, h.dim), 50.0, device=where[0], dtype=where[1])
    vc, slot, out, at = kc.clone(), torch.zeros(1, dtype=torch.long, device=where[0]), [], 0
    for n in parts:
        x = row[:, at:at + n].contiguous()
        if n == 1 and at:
            slot.fill_(at)
            out.append(ops.chunk_attention.decode(x, *w, kc, vc, h, slot, kv0, cos, sin, base=at))
        else:
            q, k, v = ops.chunk_attention.prepare(x, *w, h, kv0, cos, sin, base=at)
            out.append(ops.chunk_attention.prefill(q, k, v, kc, vc, h, kv0, base=at))
            ops.chunk_attention.store(k, v, kc, vc, h, kv0, base=at)
        at += n
    assert at == T
    return torch.cat(out, 1)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("chunk", [0, 1, 17, 64, 65, 129])
@pytest.mark.parametrize("H,G,d,rot", [(4, 2, 24, 16), (5, 5, 9, 6), (4, 1, 128, 64), (20, 1, 64, 64), (2, 2, 256, 32), (3, 1, 32, 0)])
def test_chunk_attention_alone(H, G, d, rot, chunk, where):
    """Whole prompt, portions, decode; the second row is padded (with NaN on the GPU)."""
    B, T, start, scale = 2, 290, 33, 2.0 * d ** -0.5
    row, w, h, cos, sin = _attn_case(where, H, G, d, rot, B, T, chunk, scale)
    kv0 = torch.tensor([0, start], dtype=torch.int32, device=where[0])
    if where[0] == "cuda":
        row[1, :start] = float("nan")
    want = [_attn_oracle(row[b, s:], w, h) for b, s in ((0, 0), (1, start))]
    for parts in ([T], [77, 2, 64, 130, 17], [200] + [1] * 90):
        got = _attn_run(where, row, w, h, cos, sin, kv0, parts)
        for b, s in ((0, 0), (1, start)):
            rel(got[b, s:], want[b], where, 5e-5, 0.03)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("H,G,d,rot", [(2, 1, 24, 8), (1, 1, 9, 4), (2, 2, 128, 64)])
def test_chunk_edges_and_first_key(H, G, d, rot, where):
    """One key that stands out: it takes the whole softmax up to its chunk's last position and nothing
    one position later, in prompts, portions and decoding; at position 0, at a chunk's first and last
    position, and far back in a sequence without chunks."""
    T, size = 300, 128
    for hot, chunk in ((0, size), (127, size), (128, size), (200, size), (0, 0), (64, 0)):
        row, w, h, cos, sin = _attn_case(where, H, G, d, rot, 1, T, chunk, 8.0 * d ** -0.5, seed=hot)
        zero = torch.zeros_like(w[0])
        w = (zero, torch.ones_like(w[1]), torch.ones_like(w[2]))
        # the score of the hot key: equal directions in the unrotated dimensions, opposite ones elsewhere
        u = torch.zeros(d, device=where[0], dtype=where[1])
        u[rot:] = 1.0
        row[0, :, :H * d] = u.repeat(H)
        row[0, :, H * d:] = -u.repeat(G) + 0.1 * row[0, :, H * d:]
        row[0, hot, H * d:] = u.repeat(G)
        want = _attn_oracle(row[0], w, h)
        v = f64(row)[0, hot, H * d:].view(G, d).repeat_interleave(H // G, 0).reshape(-1)
        inside = [hot, T - 1] if not chunk else [hot, hot // size * size + size - 1]
        outside = hot // size * size + size if chunk else None
        for t in inside:
            if t < T:
                assert (want[t] - v).abs().max() < 2e-2 * v.abs().max(), (hot, t)  # it does stand out
        if outside is not None and outside < T:
            assert (want[outside] - v).abs().max() > 0.5 * v.abs().max()
        tail = min(T - 1, max(inside[-1] - 1, hot + 1))
        for parts in ([T], [hot + 1, T - hot - 1], [tail] + [1] * (T - tail)):
            rel(_attn_run(where, row, w, h, cos, sin, None, parts)[0], want, where, 5e-5, 0.03)


# --------------------------------------------------------------- the framework around the model
def _greedy(cfg, P, toks, n):
    toks, margins = list(toks), []
    for _ in range(n):
        lg = O.forward(toks, P, cfg)[-1]
        top = lg.topk(2)
        margins.append((top.values[0] - top.values[1]).item() / lg.std().item())
        toks.append(int(top.indices[0]))
    return toks, margins


@pytest.mark.parametrize("where", FP32)
@pytest.mark.parametrize("name", ["mix", "odd"])
def test_greedy_generation(name, where):
    """generate(): unequal left-padded prompts, greedy, against the oracle; on the GPU also the
    captured step, replayed by a second call with other prompts of the same shape."""
    cfg, P, m = model_of(name, where)
    n = 12
    for seed in (20, 40):
        prompts = [tokens_of(cfg, k, seed + k) for k in (3, 17, 1)]
        T = max(map(len, prompts))
        ids = torch.tensor([[0] * (T - len(p)) + p for p in prompts], device=where[0])
        am = torch.tensor([[0] * (T - len(p)) + [1] * len(p) for p in prompts], device=where[0])
        for graph in ([False] if where[0] == "cpu" else [False, True, True]):
            seqs = generate(m, ids, am, max_new_tokens=n, do_sample=False, use_graph=graph)
            assert seqs.shape == (3, T + n)
            for r, p in enumerate(prompts):
                want, margins = _greedy(cfg, P, p, n)
                sure = next((i for i, g in enumerate(margins) if g < 1e-3), n)
                assert seqs[r, T:T + sure].tolist() == want[len(p):len(p) + sure]
                assert sure >= n // 2


@GPU
@pytest.mark.parametrize("B", [5, 24])
@torch.no_grad()
def test_graph_equals_eager_bf16(B):
    """The captured decode step, replayed many times, against the eager loop (same kernels)."""
    cfg, P, m = model_of("heads", ("cuda", torch.bfloat16))
    ids = torch.tensor([tokens_of(cfg, 21, s) for s in range(B)], device="cuda")
    a = generate(m, ids, max_new_tokens=60, do_sample=False, use_graph=False)
    for _ in range(3):
        torch.cuda.synchronize()
        b = generate(m, ids, max_new_tokens=60, do_sample=False, use_graph=True)
        assert torch.equal(a, b)


@pytest.mark.parametrize("where", FP32)
def test_sampling_and_mask(where):
    cfg, P, m = model_of("mix", where)
    ids = torch.tensor([tokens_of(cfg, 9), tokens_of(cfg, 9, 1)], device=where[0])
    out = [generate(m, ids, max_new_tokens=6, do_sample=True, temperature=0.9, top_p=0.9, seed=7, return_mask=True,
                    generator=torch.Generator().manual_seed(3)) for _ in range(2)]
    assert torch.equal(out[0][0], out[1][0]) and out[0][0].shape == (2, 15)
    assert out[0][1].sum() == 30 and int(out[0][0].max()) < cfg["vocab"]


def test_config_and_checkpoint_roundtrip(tmp_path):
    cfg, P, m = model_of("odd", ("cpu", torch.float32))
    back = ModelConfig.from_hf(m.cfg.to_hf())
    assert back == m.cfg and back.postln_alpha == 2.5 and back.logit_softcap == 7.0 and back.norm_eps == 1e-2
    assert ModelConfig.from_dict(json.loads(json.dumps(m.cfg.to_dict()))) == m.cfg
    assert set(m.hf_state_dict()) == set(P)
    for k, v in m.hf_state_dict().items():
        assert torch.equal(v, P[k]), k
    assert sum(v.numel() for v in P.values()) == sum(p.numel() for p in m.parameters()) == m.cfg.num_params()
    save_hf_pretrained(m, None, str(tmp_path))
    (tmp_path / "dla_config.json").unlink()  # config.json alone describes the model ...
    d = json.loads((tmp_path / "config.json").read_text())
    for e in d["layers"]:
        e["mixer"].pop("rank", None)         # ... with the sizes that only the tensors have
    (tmp_path / "config.json").write_text(json.dumps(d))
    again = load_causal_lm(str(tmp_path), gradient_checkpointing=False, device="cpu").model
    ids = torch.tensor([tokens_of(cfg, 20)])
    with torch.no_grad():
        assert torch.equal(m(ids), again(ids)) and torch.equal(m.logits(m(ids)), again.logits(again(ids)))
    sd = dict(m.hf_state_dict())
    del sd["l1.mix.a2.b"]
    with pytest.raises(KeyError):
        again.load_hf_state_dict(sd, strict=True)
    headless = load_causal_lm(str(tmp_path), gradient_checkpointing=False, device="cpu", headless=True).model
    with torch.no_grad():
        assert torch.equal(m(ids), headless(ids))


def test_meta_build_matches_and_presets():
    from distributed_llm_alignment_amd.models.materialize import materialize

    cfg = get_config("tiny-zenevik")
    a = build_model(cfg, device="cpu", seed=3)
    b = build_model(cfg, dtype=torch.float32, seed=3, meta=True)
    materialize(b, "cpu")
    for (n, p), (_, q) in zip(a.named_parameters(), b.named_parameters()):
        assert torch.equal(p, q), n
    assert (a.layers[0].ln1_w == 1).all() and (a.norm_w == 1).all() and (a.layers[1].mix.norm_w == 1).all()
    assert (a.layers[0].mix.lam < 0).all()
    assert sum(p.numel() for p in a.parameters()) == cfg.num_params()
    for name in ("zenevik-1b", "zenevik-7b"):
        c = get_config(name)
        assert c.name == name and c.num_params() > 5e8 and c.flops_per_token(2048) > 1e9


def test_serving_bench_peers():
    """The models measured beside a size have its layer count, width, heads and feed-forward parameters."""
    from distributed_llm_alignment_amd.eval import serve_bench

    for name in serve_bench.SIZES["zenevik"]:
        cfg = get_config(name)
        peers = serve_bench.peers(cfg)
        assert set(peers) == {"peer", "peer_attention"}
        for p in peers.values():
            assert p.num_layers == cfg.num_layers and p.hidden_size == cfg.hidden_size and p.vocab_size == cfg.vocab_size
            assert 0.8 < p.num_params() / cfg.num_params() < 1.2


def test_bad_configs_are_refused():
    for edit in (lambda c: c["layers"][0].update(type="retention"),
                 lambda c: c["layers"][0]["mixer"].update(blocks=7),
                 lambda c: c["layers"][1]["mixer"].pop("tau"),
                 lambda c: c["layers"][2]["mixer"].update(kv_heads=3),
                 lambda c: c["layers"][2]["mixer"].update(vdim=16),
                 lambda c: c["layers"][2]["mixer"]["rot"].update(dims=5),
                 lambda c: c["layers"][1]["mlp"].update(kind="other"),
                 lambda c: c.update(architecture="Other")):
        c = json.loads(json.dumps(CONFIGS["mix"]))
        edit(c)
        with pytest.raises(ValueError):
            ModelConfig.from_hf(c)
    with pytest.raises(ValueError):
        get_config("zenevik-1b@tp2")


def test_trains_on_cpu():
    """The PyTorch forms of the ops are differentiable: every weight gets a gradient, through the soft
    cap of the logits too."""
    m = build_model(get_config("tiny-zenevik"), device="cpu", seed=0)
    ids = torch.randint(0, 320, (2, 20))
    loss = m.causal_lm_loss(ids, ids)
    loss.backward()
    assert all(p.grad is not None and torch.isfinite(p.grad).all() for p in m.parameters())
    with torch.no_grad():
        lp = torch.log_softmax(m.logits(m(ids)), -1)[:, :-1].gather(-1, ids[:, 1:, None])
    assert abs(loss.item() + lp.mean().item()) < 1e-5


@GPU
def test_gpu_training_is_refused():
    m = build_model(get_config("tiny-zenevik"), device="cuda", seed=0)
    with pytest.raises(NotImplementedError):
        m(torch.zeros(1, 4, dtype=torch.long, device="cuda"))


@pytest.mark.parametrize("where", WHERE)
def test_trace_runner(where):
    """Batches that start together and end one by one; wanted places in prompts and decoded."""
    cfg, P, m = model_of("mix", where)
    r = TraceRunner(m, 400)
    plan = {"a": (1, 3), "b": (70, 20), "c": (9, 11)}
    seqs = {i: tokens_of(cfg, n + k, 50 + n) for i, (n, k) in plan.items()}
    want_first = {"a": [0], "b": [69, 0, 33], "c": []}
    out = r.step([{"id": i, "tokens": seqs[i][:n], "want": want_first[i]} for i, (n, _) in plan.items()], [])
    ref = torch.cat([want_of(cfg, P, seqs[i])[want_first[i]] for i in plan if want_first[i]])
    close(out, ref, where)
    for t in range(20):
        live = [i for i, (n, k) in plan.items() if t < k]
        ent = [{"id": i, "tokens": [seqs[i][plan[i][0] + t]], "want": [0] if t % 2 else []} for i in reversed(live)]
        out = r.step(ent, [i for i in live if t + 1 == plan[i][1]])
        if t % 2 == 0:
            assert out is None
        else:
            close(out, torch.stack([want_of(cfg, P, seqs[i])[plan[i][0] + t] for i in reversed(live)]), where)
    assert not r.where


def test_trace_run_program(tmp_path):
    cfg, P, m = model_of("min", ("cpu", torch.float32))
    save_hf_pretrained(m, None, str(tmp_path / "model"))
    (tmp_path / "out").mkdir()
    toks = tokens_of(cfg, 12)
    steps = [{"step": 0, "entries": [{"id": "q", "tokens": toks[:11], "want": [3, 10]}], "end": []},
             {"step": 1, "entries": [{"id": "q", "tokens": toks[11:], "want": [0]}], "end": ["q"]}]
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "model"), "--dtype", "float32",
                        "--out", str(tmp_path / "out"), "--max-tokens", "16", "--device", "cpu"], text=True,
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, timeout=300,
                       env={**os.environ, "PATH": os.path.dirname(sys.executable) + os.pathsep + os.environ.get("PATH", "")})
    assert p.returncode == 0, p.stderr[-2000:]
    want = want_of(cfg, P, toks)
    for name, places in (("0.f32", [3, 10]), ("1.f32", [11])):
        got = torch.frombuffer(bytearray((tmp_path / "out" / name).read_bytes()), dtype=torch.float32).view(len(places), -1)
        close(got, want[places], ("cpu", torch.float32))


def test_parallel_forms_and_fp8_are_refused():
    from distributed_llm_alignment_amd.parallel.layer_split import dispatch_layers
    from distributed_llm_alignment_amd.parallel.tensor_parallel import apply_tensor_parallel

    m = build_model(get_config("tiny-zenevik"), device="cpu", seed=0)
    with pytest.raises(NotImplementedError):
        apply_tensor_parallel(m, None, tp_rank=0, tp_size=2)
    with pytest.raises(NotImplementedError):
        dispatch_layers(m, ["cpu", "cpu"])
    with pytest.raises(ValueError):
        generate(m, torch.zeros(1, 3, dtype=torch.long), max_new_tokens=2, weight_dtype="fp8")


def test_teacher_generation_program(tmp_path):
    """The command line around generate() takes the design by preset name."""
    from distributed_llm_alignment_amd.training.generate_teacher_data import main

    (tmp_path / "p.jsonl").write_text("".join(json.dumps({"prompt": t}) + "\n" for t in ("a", "some longer prompt")))
    assert main(["--teacher", "tiny-zenevik", "--prompts", str(tmp_path / "p.jsonl"), "--output", str(tmp_path / "o.jsonl"),
                 "--batch_size", "2", "--max_new_tokens", "5"]) == 0
    assert len((tmp_path / "o.jsonl").read_text().splitlines()) == 2
