"""Plain, slow Zenevik in float64 on the CPU: the oracle the framework is compared with.

One function per mechanism, written from the design's equations, token by token where that is the
plainest form. Shares no code with the package. `P` is a dict of tensors by checkpoint name, `cfg`
the parsed config.json. Everything takes ONE sequence: x is [T, width], positions are 0 .. T-1.
"""
import math

import torch

from vufilorn_oracle import F64, gelu_tanh, rms, rotate, silu


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def log_sigmoid(z):
    return -softplus(-z)


# ------------------------------------------------------------------------- gated linear recurrence
def causal_conv(x, w, b):
    """x [T, C], w [C, taps] (last column: the current token), zeros before the start."""
    T, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x) + b
    for t in range(T):
        for j in range(taps):
            if t - j >= 0:
                out[t] = out[t] + w[:, taps - 1 - j] * x[t - j]
    return out


def block_gate(u, w, b):
    """sigmoid of a block-diagonal product: w [blocks, n, n] (out, in), b [blocks, n]."""
    T, nb = u.shape[0], w.shape[0]
    parts = u.view(T, nb, -1)
    return sigmoid(torch.stack([parts[:, i] @ w[i].T + b[i] for i in range(nb)], 1)).reshape(T, -1)


def lru_scan(u, r, i, lam, S=None):
    """S_t = a S_(t-1) + sqrt(1 - a^2) i u with log a = -8 r softplus(lam); returns all S_t."""
    S = torch.zeros(u.shape[1], dtype=F64) if S is None else S
    out = []
    for t in range(u.shape[0]):
        a = torch.exp(-8.0 * r[t] * softplus(lam))
        S = a * S + torch.sqrt(1.0 - a * a) * i[t] * u[t]
        out.append(S)
    return torch.stack(out)


def rglru(h, P, pre):
    y = gelu_tanh(h @ P[pre + "y"].T + P[pre + "y.b"])
    u = causal_conv(h @ P[pre + "x"].T + P[pre + "x.b"], P[pre + "conv"], P[pre + "conv.b"])
    r = block_gate(u, P[pre + "ra"], P[pre + "ra.b"])
    i = block_gate(u, P[pre + "ri"], P[pre + "ri.b"])
    return (lru_scan(u, r, i, P[pre + "lam"]) * y) @ P[pre + "o"].T


# ------------------------------------------------------------------------- gated linear attention
def gla_recurrence(q, k, v, log_alpha, S=None):
    """q, k, log_alpha [T, heads, dim], v [T, heads, vdim]: per head S = diag(alpha) S + k v^T,
    o = S^T q. Returns (o [T, heads, vdim], final S [heads, dim, vdim])."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=F64) if S is None else S
    out = []
    for t in range(T):
        S = torch.exp(log_alpha[t])[:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def gla(h, P, pre, m, eps):
    T, H, d, vd = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ P[pre + "q"].T).view(T, H, d) * d ** -0.5
    k = (h @ P[pre + "k"].T).view(T, H, d)
    v = (h @ P[pre + "v"].T).view(T, H, vd)
    z = (h @ P[pre + "a1"].T) @ P[pre + "a2"].T + P[pre + "a2.b"]
    o, _ = gla_recurrence(q, k, v, log_sigmoid(z).view(T, H, d) / m["tau"])
    o = (rms(o, eps) * P[pre + "norm"]).reshape(T, H * vd)
    return (o * silu(h @ P[pre + "g"].T)) @ P[pre + "o"].T


# ------------------------------------------------------------------------------ chunked attention
def chunk_softmax(scores, size):
    """scores [T, T] -> weights: query i sees keys j <= i of its own chunk of `size` positions."""
    T = scores.shape[0]
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    ok = j <= i
    if size:
        ok = ok & (i // size == j // size)
    return torch.softmax(scores.masked_fill(~ok, float("-inf")), -1)


def attend(q, k, v, scale, size):
    """q [T, H, d], k [T, G, d], v [T, G, vd] -> [T, H, vd]; query head n reads key head n // (H / G)."""
    H, G = q.shape[1], k.shape[1]
    return torch.stack([chunk_softmax(q[:, n] @ k[:, n // (H // G)].T * scale, size) @ v[:, n // (H // G)]
                        for n in range(H)], 1)


def attention(h, P, pre, m, eps):
    T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = h @ P[pre + "q"].T + P[pre + "q.b"]
    k = h @ P[pre + "k"].T + P[pre + "k.b"]
    v = k.view(T, G, d)  # the values are the projected keys themselves
    q = (rms(q, eps) * P[pre + "q.norm"]).view(T, H, d)
    k = (rms(k, eps) * P[pre + "k.norm"]).view(T, G, d)
    q = rotate(q, m["rot"]["base"], m["rot"]["dims"])
    k = rotate(k, m["rot"]["base"], m["rot"]["dims"])
    o = attend(q, k, v, m["scale"], (m.get("mask") or {}).get("size", 0))
    return o.reshape(T, H * d) @ P[pre + "o"].T + P[pre + "o.b"]


# -------------------------------------------------------------------------------------- the model
def feed_forward(h, P, pre):
    return (gelu_tanh(h @ P[pre + "gate"].T) * (h @ P[pre + "up"].T)) @ P[pre + "down"].T


def run_layer(x, P, cfg, i):
    """Norm after the sum: x <- rms(alpha x + sublayer(x)) * w, twice."""
    spec, eps, pre, alpha = cfg["layers"][i], cfg["norm"]["eps"], f"l{i}.", cfg["postln_alpha"]
    if spec["type"] == "rglru":
        y = rglru(x, P, pre + "mix.")
    elif spec["type"] == "gla":
        y = gla(x, P, pre + "mix.", spec["mixer"], eps)
    else:
        y = attention(x, P, pre + "mix.", spec["mixer"], eps)
    x = rms(alpha * x + y, eps) * P[pre + "norm1"]
    if spec.get("mlp"):
        x = rms(alpha * x + feed_forward(x, P, pre + "mlp."), eps) * P[pre + "norm2"]
    return x


def softcap(z, cap):
    return cap * torch.tanh(z / cap)


def forward(tokens, P, cfg, layers_out=None):
    """Logits [T, vocab] of one sequence; `layers_out` (a list) collects x after every layer."""
    P = {k: (v.to(F64) if v.is_floating_point() else v) for k, v in P.items()}
    x = P["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i in range(len(cfg["layers"])):
        x = run_layer(x, P, cfg, i)
        if layers_out is not None:
            layers_out.append(x)
    return softcap((rms(x, cfg["norm"]["eps"]) * P["final.norm"]) @ P["head"].T, cfg["logit_softcap"])


# ------------------------------------------------------------------ small random models for tests
def lru(width, blocks, conv):
    return {"width": width, "blocks": blocks, "conv": conv}


def gated(heads, dim, vdim, tau, rank):
    """`rank` (of the decay's two projections) is a tensor shape, not a config entry: see config()."""
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau, "rank": rank}


def attn(heads, kv_heads, dim, rot, size, scale, base=10000.0):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "rot": {"base": base, "dims": rot},
            "mask": {"size": size}, "scale": scale}


def kind_of(m):
    return "rglru" if "blocks" in m else "gla" if "tau" in m else "attention"


def config(width, vocab, layers, alpha=2.0, cap=20.0, eps=1e-5):
    """layers: [(mixer dict, ff or None)]."""
    return {"architecture": "Zenevik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "postln_alpha": alpha,
            "logit_softcap": cap, "layers": [{"type": kind_of(m), "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}
                                             for m, ff in layers]}


def weights(cfg, seed=0, gain=1.6):
    """Random checkpoint tensors of cfg, rounded to bfloat16 values, as float32."""
    g = torch.Generator().manual_seed(seed)
    P = {}

    def mat(name, *shape, gn=gain):
        P[name] = torch.randn(*shape, generator=g) * gn / math.sqrt(shape[-1])

    def vec(name, *shape, mean=0.0, std=0.3):
        P[name] = mean + std * torch.randn(*shape, generator=g)

    H, V = cfg["width"], cfg["vocab"]
    P["embed"] = torch.randn(V, H, generator=g)
    for i, e in enumerate(cfg["layers"]):
        m, p = e["mixer"], f"l{i}.mix."
        vec(f"l{i}.norm1", H, mean=1.0)
        if e["type"] == "rglru":
            W, nb, n = m["width"], m["blocks"], m["width"] // m["blocks"]
            for t in ("y", "x"):
                mat(p + t, W, H)
                vec(p + t + ".b", W)
            vec(p + "conv", W, m["conv"], std=0.6)
            vec(p + "conv.b", W)
            for t, mean, std in (("ra", -2.0, 2.5), ("ri", 0.0, 1.0)):
                mat(p + t, nb, n, n)
                vec(p + t + ".b", nb, n, mean=mean, std=std)
            vec(p + "lam", W, mean=-2.0, std=1.5)
            mat(p + "o", H, W)
        elif e["type"] == "gla":
            n = m["heads"]
            for t, k in (("q", m["dim"]), ("k", m["dim"]), ("v", m["vdim"]), ("g", m["vdim"])):
                mat(p + t, n * k, H)
            mat(p + "a1", m["rank"], H)
            mat(p + "a2", n * m["dim"], m["rank"])
            vec(p + "a2.b", n * m["dim"], mean=2.0, std=2.0)
            vec(p + "norm", m["vdim"], mean=1.0)
            mat(p + "o", H, n * m["vdim"])
        else:
            for t, k in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"])):
                mat(p + t, k, H)
                vec(p + t + ".b", k)
                vec(p + t + ".norm", k, mean=1.0)
            mat(p + "o", H, m["heads"] * m["dim"])
            vec(p + "o.b", H)
        if e["mlp"]:
            vec(f"l{i}.norm2", H, mean=1.0)
            mat(f"l{i}.mlp.gate", e["mlp"]["ff"], H)
            mat(f"l{i}.mlp.up", e["mlp"]["ff"], H)
            mat(f"l{i}.mlp.down", H, e["mlp"]["ff"])
    vec("final.norm", H, mean=1.0)
    mat("head", V, H)
    return {k: v.bfloat16().float() for k, v in P.items()}
