"""Per-layer design specs (`ModelConfig.layer_specs`): validation, parameter and FLOP counts.

A spec is {"type": mixer name, "mixer": {sizes and constants}, "mlp": {"kind", "ff"} or None}. The
modules built from it live in models/mixers.py.
"""
from __future__ import annotations

from typing import Any, Dict

_MIXER_KEYS = {
    "latent_attention": ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank", "rot", "scale"),
    "retention": ("heads", "dim", "vdim", "rot", "decay"),
}


def check_spec(spec: Dict[str, Any], i: int) -> None:
    """Raise ValueError for a layer spec no module implements."""
    kind = spec.get("type")
    if kind not in _MIXER_KEYS:
        raise ValueError(f"layer {i}: unknown mixer type {kind!r} (have {sorted(_MIXER_KEYS)})")
    m = spec["mixer"]
    missing = [k for k in _MIXER_KEYS[kind] if k not in m]
    if missing:
        raise ValueError(f"layer {i} ({kind}): config lacks {missing}")
    dims = m["rot"]["dims"]
    if dims % 2 or not 0 <= dims <= (m["rot_dim"] if kind == "latent_attention" else m["dim"]):
        raise ValueError(f"layer {i} ({kind}): rot.dims {dims} is odd or wider than the rotated vector")
    if kind == "latent_attention" and dims != m["rot_dim"]:
        raise ValueError(f"layer {i}: rot.dims {dims} != rot_dim {m['rot_dim']}")
    if kind == "retention" and len(m["decay"]) != m["heads"]:
        raise ValueError(f"layer {i}: {len(m['decay'])} decays for {m['heads']} heads")
    mlp = spec.get("mlp")
    if mlp and mlp.get("kind", "dense") != "dense":
        raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")


def window(mixer: Dict[str, Any]) -> int:
    """Sliding-window size of a latent-attention mixer (0: all earlier tokens)."""
    return int((mixer.get("mask") or {}).get("size", 0) or 0)


def _matmul_params(cfg, i: int) -> int:
    spec, H = cfg.layer_specs[i], cfg.hidden_size
    m = spec["mixer"]
    n = m["heads"]
    if spec["type"] == "latent_attention":
        p = H * (m["q_rank"] + m["kv_rank"] + m["rot_dim"]) + n * (m["dim"] + m["rot_dim"]) * m["q_rank"]
        p += n * (m["dim"] + m["vdim"]) * m["kv_rank"] + n * m["vdim"] * H
    else:
        p = 2 * n * (m["dim"] + m["vdim"]) * H + n * m["vdim"] * H
    if spec.get("mlp"):
        p += 2 * H * spec["mlp"]["ff"]
    return p + 2 * H * cfg.token_side_dim


def spec_param_count(cfg, i: int) -> int:
    spec, H = cfg.layer_specs[i], cfg.hidden_size
    m = spec["mixer"]
    n = _matmul_params(cfg, i) + H * (1 + bool(spec.get("mlp")) + bool(cfg.token_side_dim))
    return n + (m["q_rank"] + m["kv_rank"] if spec["type"] == "latent_attention" else 0)


def spec_flops_per_token(cfg, i: int, seq_len: int) -> float:
    """Forward FLOPs of one run of layer i per token: matmuls plus the mixer's token mixing
    (mean visible keys under the window; the recurrence's state update and read)."""
    m = cfg.layer_specs[i]["mixer"]
    n, f = m["heads"], 2.0 * _matmul_params(cfg, i)
    if cfg.layer_specs[i]["type"] == "latent_attention":
        w = window(m)
        keys = seq_len / 2 if not w or w >= seq_len else w - w * w / (2.0 * seq_len)
        return f + 2.0 * n * (m["dim"] + m["rot_dim"] + m["vdim"]) * keys
    return f + 4.0 * n * m["dim"] * m["vdim"]
