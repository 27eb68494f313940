"""Per-layer design specs (`ModelConfig.layer_specs`): validation, parameter and FLOP counts.

A spec is {"type": mixer name, "mixer": {sizes and constants}, "mlp": {"kind", "ff"} or None}. The
modules built from it live in models/mixers.py.
"""
from __future__ import annotations

from typing import Any, Dict, List, Sequence

_MIXER_KEYS = {
    "latent_attention": ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank", "rot", "scale"),
    "retention": ("heads", "dim", "vdim", "rot", "decay"),
    "rglru": ("width", "blocks", "conv"),
    "gla": ("heads", "dim", "vdim", "tau"),
    "attention": ("heads", "kv_heads", "dim", "vdim", "rot", "scale"),
}

# sizes that config.json may leave to a tensor's shape: (key, tensor, axis) per mixer
TENSOR_SIZES = {"gla": (("rank", "mix.a1", 0),)}
_DEFAULT_RANK = 16


def checked_specs(layers: List[Dict[str, Any]], types: Sequence[str]) -> List[Dict[str, Any]]:
    """The layer specs of a config.json after validation (`types`: the mixers the design has)."""
    specs = [dict(e) for e in layers]
    for i, e in enumerate(specs):
        if e.get("type") not in types:
            raise ValueError(f"layer {i}: unknown mixer type {e.get('type')!r} (have {sorted(types)})")
        check_spec(e, i)
    return specs


def check_spec(spec: Dict[str, Any], i: int) -> None:
    """Raise ValueError for a layer spec no module implements."""
    kind = spec.get("type")
    if kind not in _MIXER_KEYS:
        raise ValueError(f"layer {i}: unknown mixer type {kind!r} (have {sorted(_MIXER_KEYS)})")
    m = spec["mixer"]
    missing = [k for k in _MIXER_KEYS[kind] if k not in m]
    if missing:
        raise ValueError(f"layer {i} ({kind}): config lacks {missing}")
    if "rot" in m:
        dims = m["rot"]["dims"]
        if dims % 2 or not 0 <= dims <= (m["rot_dim"] if kind == "latent_attention" else m["dim"]):
            raise ValueError(f"layer {i} ({kind}): rot.dims {dims} is odd or wider than the rotated vector")
    if kind == "latent_attention" and dims != m["rot_dim"]:
        raise ValueError(f"layer {i}: rot.dims {dims} != rot_dim {m['rot_dim']}")
    if kind == "retention" and len(m["decay"]) != m["heads"]:
        raise ValueError(f"layer {i}: {len(m['decay'])} decays for {m['heads']} heads")
    if kind == "rglru" and (m["width"] % m["blocks"] or m["conv"] < 1):
        raise ValueError(f"layer {i}: width {m['width']} in {m['blocks']} blocks, {m['conv']} taps")
    if kind == "gla" and not m["tau"] > 0:
        raise ValueError(f"layer {i}: tau {m['tau']}")
    if kind == "attention":
        if m["heads"] % m["kv_heads"]:
            raise ValueError(f"layer {i}: {m['heads']} query heads on {m['kv_heads']} key heads")
        if m["vdim"] != m["dim"]:
            raise ValueError(f"layer {i}: the values are the keys, but vdim {m['vdim']} != dim {m['dim']}")
    mlp = spec.get("mlp")
    if mlp and mlp.get("kind", "dense") != "dense":
        raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")


def window(mixer: Dict[str, Any]) -> int:
    """The mask's size (sliding window of a latent-attention mixer, chunk of an attention mixer); 0: all
    earlier tokens."""
    return int((mixer.get("mask") or {}).get("size", 0) or 0)


def decay_rank(mixer: Dict[str, Any]) -> int:
    """Rank of a gated-linear-attention mixer's two decay projections."""
    return int(mixer.get("rank", _DEFAULT_RANK))


def _mixer_params(kind: str, m: Dict[str, Any], H: int):
    """(parameters in matrix products, the other parameters) of one mixer."""
    n = m.get("heads", 0)
    if kind == "latent_attention":
        p = H * (m["q_rank"] + m["kv_rank"] + m["rot_dim"]) + n * (m["dim"] + m["rot_dim"]) * m["q_rank"]
        return p + n * (m["dim"] + m["vdim"]) * m["kv_rank"] + n * m["vdim"] * H, m["q_rank"] + m["kv_rank"]
    if kind == "retention":
        return 2 * n * (m["dim"] + m["vdim"]) * H + n * m["vdim"] * H, 0
    if kind == "rglru":
        W = m["width"]
        return 3 * H * W + 2 * W * (W // m["blocks"]), W * (m["conv"] + 6)
    if kind == "gla":
        r = decay_rank(m)
        return 2 * n * (m["dim"] + m["vdim"]) * H + n * m["vdim"] * H + r * (H + n * m["dim"]), n * m["dim"] + m["vdim"]
    k = (n + m["kv_heads"]) * m["dim"]
    return H * k + H * n * m["vdim"], 2 * k + H


def _matmul_params(cfg, i: int) -> int:
    spec, H = cfg.layer_specs[i], cfg.hidden_size
    p = _mixer_params(spec["type"], spec["mixer"], H)[0]
    if spec.get("mlp"):
        p += (3 if cfg.activation in ("swiglu", "geglu") else 2) * H * spec["mlp"]["ff"]
    return p + 2 * H * cfg.token_side_dim


def spec_param_count(cfg, i: int) -> int:
    spec, H = cfg.layer_specs[i], cfg.hidden_size
    n = _matmul_params(cfg, i) + H * (1 + bool(spec.get("mlp")) + bool(cfg.token_side_dim))
    return n + _mixer_params(spec["type"], spec["mixer"], H)[1]


def spec_flops_per_token(cfg, i: int, seq_len: int) -> float:
    """Forward FLOPs of one run of layer i per token: matmuls plus the mixer's token mixing
    (mean visible keys under the mask; the recurrence's state update and read)."""
    kind, m = cfg.layer_specs[i]["type"], cfg.layer_specs[i]["mixer"]
    f, w = 2.0 * _matmul_params(cfg, i), window(m)
    if kind == "latent_attention":
        keys = seq_len / 2 if not w or w >= seq_len else w - w * w / (2.0 * seq_len)
        return f + 2.0 * m["heads"] * (m["dim"] + m["rot_dim"] + m["vdim"]) * keys
    if kind == "attention":
        return f + 2.0 * m["heads"] * (m["dim"] + m["vdim"]) * (min(seq_len, w) if w else seq_len) / 2
    return f + (4.0 * m["heads"] * m["dim"] * m["vdim"] if kind != "rglru" else 4.0 * m["width"])
