"""Plain, slow Vufilorn in float64 on the CPU: the oracle the framework is compared with.

One function per mechanism, written from the design's equations, token by token where that is the
plainest form. Shares no code with the package. `P` is a dict of tensors by checkpoint name, `cfg`
the parsed config.json. Everything takes ONE sequence: x is [T, width], positions are 0 .. T-1.
"""
import math

import torch

F64 = torch.float64


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z / (1.0 + torch.exp(-z))


def rotate(x, base, dims, pos0=0):
    """Rotary positions on x [T, heads, D]: dimension i pairs with i + dims/2 for i < dims/2."""
    T, half = x.shape[0], dims // 2
    out = x.clone()
    for i in range(half):
        f = float(base) ** (-2.0 * i / dims)
        a = (torch.arange(T, dtype=F64) + pos0) * f
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[:, :, i], x[:, :, i + half]
        out[:, :, i] = u * c - v * s
        out[:, :, i + half] = v * c + u * s
    return out


def window_softmax(scores, size):
    """scores [T, T] -> weights: query i sees keys j with 0 <= i - j < size (size 0: all j <= i)."""
    T = scores.shape[0]
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    ok = j <= i
    if size:
        ok = ok & (i - j < size)
    return torch.softmax(scores.masked_fill(~ok, float("-inf")), -1)


def latent_attention(h, P, pre, m, eps):
    T, H, d, r, vd, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    cq = rms(h @ P[pre + "dq"].T, eps) * P[pre + "dq.norm"]
    q = (cq @ P[pre + "uq"].T).view(T, H, d + r)
    down = h @ P[pre + "dkv"].T
    c = rms(down[:, :R], eps) * P[pre + "dkv.norm"]
    base = m["rot"]["base"]
    qr = rotate(q[:, :, d:], base, r)
    kr = rotate(down[:, None, R:], base, r)[:, 0]
    kn = (c @ P[pre + "uk"].T).view(T, H, d)
    v = (c @ P[pre + "uv"].T).view(T, H, vd)
    size = (m.get("mask") or {}).get("size", 0)
    heads = []
    for n in range(H):
        s = (q[:, n, :d] @ kn[:, n].T + qr[:, n] @ kr.T) * m["scale"]
        heads.append(window_softmax(s, size) @ v[:, n])
    return torch.cat(heads, -1) @ P[pre + "o"].T


def retention(h, P, pre, m, eps, state=None, pos0=0):
    """Returns (output, final state [heads, dim, vdim]); `state` / `pos0` continue a sequence."""
    T, H, d, vd = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = rotate((h @ P[pre + "q"].T).view(T, H, d), m["rot"]["base"], m["rot"]["dims"], pos0)
    k = rotate((h @ P[pre + "k"].T).view(T, H, d), m["rot"]["base"], m["rot"]["dims"], pos0) * d ** -0.5
    v = (h @ P[pre + "v"].T).view(T, H, vd)
    dec = torch.tensor(m["decay"], dtype=F64)[:, None, None]
    S = torch.zeros(H, d, vd, dtype=F64) if state is None else state
    out = torch.empty(T, H, vd, dtype=F64)
    for t in range(T):
        S = dec * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    y = rms(out, eps).reshape(T, H * vd) * silu(h @ P[pre + "g"].T)
    return y @ P[pre + "o"].T, S


def feed_forward(h, P, pre):
    return torch.relu(h @ P[pre + "up"].T) ** 2 @ P[pre + "down"].T


def side_input(x, tokens, P, layer, dim, eps):
    pre = f"l{layer}.side."
    e = P["side.embed"][tokens][:, layer * dim:(layer + 1) * dim]
    g = gelu_tanh(x @ P[pre + "gate"].T) * e
    return x + rms(g @ P[pre + "proj"].T, eps) * P[pre + "norm"]


def run_layer(x, tokens, P, cfg, i):
    spec, eps, pre = cfg["layers"][i], cfg["norm"]["eps"], f"l{i}."
    h = rms(x, eps) * (1.0 + P[pre + "norm1"])
    if spec["type"] == "latent_attention":
        x = x + latent_attention(h, P, pre + "mix.", spec["mixer"], eps)
    else:
        x = x + retention(h, P, pre + "mix.", spec["mixer"], eps)[0]
    if spec.get("mlp"):
        x = x + feed_forward(rms(x, eps) * (1.0 + P[pre + "norm2"]), P, pre + "mlp.")
    if cfg.get("token_side"):
        x = side_input(x, tokens, P, i, cfg["token_side"]["dim"], eps)
    return x


def layer_runs(cfg):
    """[(layer, embedding output is added first)] in the order the layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    runs = [(i, False) for i in range(a)]
    for p in range(loop["times"]):
        runs += [(i, p > 0 and i == a) for i in range(a, b)]
    return runs + [(i, False) for i in range(b, n)]


def forward(tokens, P, cfg, layers_out=None):
    """Logits [T, vocab] of one sequence; `layers_out` (a list) collects x after every layer run."""
    P = {k: (v.to(F64) if v.is_floating_point() else v) for k, v in P.items()}
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    x0 = P["embed"][tokens] * cfg["embedding"]["scale"]
    x = x0
    for i, add in layer_runs(cfg):
        x = run_layer(x + x0 if add else x, tokens, P, cfg, i)
        if layers_out is not None:
            layers_out.append(x)
    return (rms(x, cfg["norm"]["eps"]) * (1.0 + P["final.norm"])) @ P["embed"].T


# ------------------------------------------------------------------ small random models for tests
def latent(heads, dim, rot, vdim, kv_rank, q_rank, scale, size, base=10000.0):
    return {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
            "scale": scale, "rot": {"base": base, "dims": rot}, "mask": {"size": size}}


def ret(heads, dim, vdim, rot, decay, base=10000.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "rot": {"base": base, "dims": rot}, "decay": decay}


def config(width, vocab, layers, side=8, scale=3.0, loop=None, eps=1e-5):
    """layers: [(mixer dict, ff or None)]."""
    return {"architecture": "Vufilorn", "vocab": vocab, "width": width, "embedding": {"scale": scale},
            "norm": {"eps": eps}, "loop": loop, "token_side": {"dim": side} if side else None,
            "layers": [{"type": "latent_attention" if "kv_rank" in m else "retention", "mixer": m,
                        "mlp": {"kind": "dense", "ff": ff} if ff else None} for m, ff in layers]}


def weights(cfg, seed=0, gain=1.6):
    """Random checkpoint tensors of cfg, rounded to bfloat16 values, as float32."""
    g = torch.Generator().manual_seed(seed)
    P = {}

    def mat(name, o, i, gn=gain):
        P[name] = torch.randn(o, i, generator=g) * gn / math.sqrt(i)

    def vec(name, n, mean):
        P[name] = mean + 0.3 * torch.randn(n, generator=g)

    H, V = cfg["width"], cfg["vocab"]
    P["embed"] = torch.randn(V, H, generator=g) * 0.3
    side = (cfg.get("token_side") or {}).get("dim", 0)
    if side:
        P["side.embed"] = torch.randn(V, len(cfg["layers"]) * side, generator=g)
    for i, e in enumerate(cfg["layers"]):
        m, p = e["mixer"], f"l{i}."
        vec(p + "norm1", H, 0.0)
        n = m["heads"]
        if e["type"] == "latent_attention":
            mat(p + "mix.dq", m["q_rank"], H)
            vec(p + "mix.dq.norm", m["q_rank"], 1.0)
            mat(p + "mix.uq", n * (m["dim"] + m["rot_dim"]), m["q_rank"])
            mat(p + "mix.dkv", m["kv_rank"] + m["rot_dim"], H)
            vec(p + "mix.dkv.norm", m["kv_rank"], 1.0)
            mat(p + "mix.uk", n * m["dim"], m["kv_rank"])
            mat(p + "mix.uv", n * m["vdim"], m["kv_rank"])
        else:
            for t, k in (("q", m["dim"]), ("k", m["dim"]), ("v", m["vdim"]), ("g", m["vdim"])):
                mat(p + "mix." + t, n * k, H)
        mat(p + "mix.o", H, n * m["vdim"])
        if e["mlp"]:
            vec(p + "norm2", H, 0.0)
            mat(p + "mlp.up", e["mlp"]["ff"], H)
            mat(p + "mlp.down", H, e["mlp"]["ff"])
        if side:
            mat(p + "side.gate", side, H)
            mat(p + "side.proj", H, side)
            vec(p + "side.norm", H, 1.0)
    vec("final.norm", H, 0.0)
    return {k: v.bfloat16().float() for k, v in P.items()}
