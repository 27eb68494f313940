"""Prefill and decode throughput of a per-layer design beside its closest models at equal size
(random weights): `python bench.py --serve vufilorn`, `python bench.py --serve zenevik`.

Every design is measured beside a Mistral (sliding window, SwiGLU) with as many layers as the design
has layer runs, the same width, heads x head size, window and vocabulary, and the feed-forward width
that gives it the same feed-forward parameters; Zenevik also beside a Vufilorn with retention where it
has a recurrent mixer and latent attention where it has attention. All run through `KVCache` and
`CausalLM`; decode is the captured step of `generate`. One JSON line per size, nothing else on stdout.
"""
from __future__ import annotations

import json
import time
from typing import Dict, List

import torch

from ..models import build_model, generate, get_config
from ..models.config import ModelConfig
from ..models.generation import KVCache, clear_graph_cache

SIZES = {"vufilorn": ("vufilorn-1b", "vufilorn-7b"), "zenevik": ("zenevik-1b", "zenevik-7b")}
PREFILL = ((1, 4096), (8, 1024))  # (batch, prompt)
DECODE = ((1, 2048), (8, 2048), (32, 512))  # (batch, prompt); 64 new tokens


def peer_config(cfg: ModelConfig, runs: int) -> ModelConfig:
    """The Mistral beside a per-layer design."""
    mix = next(e["mixer"] for e in cfg.layer_specs if e["type"] in ("latent_attention", "attention"))
    ff = cfg.layer_specs[0]["mlp"]["ff"]
    if cfg.activation == "relu2":  # two matrices against three
        ff = (ff * 2 // 3 + 1023) // 1024 * 1024
    return ModelConfig(arch="mistral", vocab_size=cfg.vocab_size, hidden_size=cfg.hidden_size, num_layers=runs,
                       num_heads=mix["heads"], num_kv_heads=mix.get("kv_heads", mix["heads"] // 4), head_dim=mix["dim"],
                       intermediate_size=ff, sliding_window=(mix.get("mask") or {}).get("size", 0), rope_theta=10000.0,
                       max_position_embeddings=8192, name=f"mistral-like-{cfg.name}")


def design_peer_config(cfg: ModelConfig) -> ModelConfig:
    """The Vufilorn beside a Zenevik: the same layer count, width, head sizes, window, vocabulary and
    feed-forward parameters, no loop and no token input."""
    like = get_config("vufilorn-1b").layer_specs[0]["mixer"]
    gla = next(e["mixer"] for e in cfg.layer_specs if e["type"] == "gla")
    att = next(e["mixer"] for e in cfg.layer_specs if e["type"] == "attention")
    lat = dict(like, heads=att["heads"], dim=att["dim"], vdim=att["vdim"], mask=att["mask"], q_rank=3 * cfg.hidden_size // 8,
               scale=(att["dim"] + like["rot_dim"]) ** -0.5)
    ret = dict(heads=gla["heads"], dim=gla["dim"], vdim=gla["vdim"], rot=dict(base=1e6, dims=gla["dim"]),
               decay=[1 - 2.0 ** -(5 + 4 * h / gla["heads"]) for h in range(gla["heads"])])
    layers = [{"type": "latent_attention" if e["type"] == "attention" else "retention",
               "mixer": lat if e["type"] == "attention" else ret,
               "mlp": {"kind": "dense", "ff": e["mlp"]["ff"] * 3 // 2}} for e in cfg.layer_specs]
    peer = ModelConfig.from_hf({"architecture": "Vufilorn", "vocab": cfg.vocab_size, "width": cfg.hidden_size,
                                "norm": {"eps": cfg.norm_eps}, "layers": layers})
    peer.name = f"vufilorn-like-{cfg.name}"
    return peer


def peers(cfg: ModelConfig) -> Dict[str, ModelConfig]:
    runs = len(cfg.layer_schedule)
    if cfg.arch == "zenevik":
        return {"peer": design_peer_config(cfg), "peer_attention": peer_config(cfg, runs)}
    return {"peer": peer_config(cfg, runs)}


def _time(fn, warm: int = 2, reps: int = 5) -> float:
    for _ in range(warm):
        fn()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(reps):
        fn()
    torch.cuda.synchronize()
    return (time.perf_counter() - t0) / reps


@torch.no_grad()
def measure(cfg: ModelConfig, what=("prefill", "decode"), seed: int = 0) -> Dict[str, float]:
    model = build_model(cfg, device="cuda", dtype=torch.bfloat16, seed=seed).eval()
    out: Dict[str, float] = {"params_b": round(sum(p.numel() for p in model.parameters()) / 1e9, 3)}
    if "prefill" in what:
        for B, T in PREFILL:
            ids = torch.randint(0, cfg.vocab_size, (B, T), device="cuda")
            cache = KVCache(model, B, T, None)

            def step():
                cache.reset(None)
                model.logits(model(ids, cache=cache)[:, -1])

            dt = _time(step)
            out[f"prefill_b{B}_t{T}_tok_s"] = round(B * T / dt)
            out[f"prefill_b{B}_t{T}_tflops"] = round(B * T * cfg.flops_per_token(T) / dt / 1e12, 1)
            del cache
    if "decode" in what:
        for B, T in DECODE:
            ids = torch.randint(0, cfg.vocab_size, (B, T), device="cuda")

            def gen(n):
                return _time(lambda: generate(model, ids, max_new_tokens=n, do_sample=False, eos_token_id=-1,
                                              pad_token_id=0, use_graph=True), 1, 2)

            # (the difference of two lengths: the prompt and the eager first steps drop out)
            per = (gen(80) - gen(16)) / 64
            out[f"decode_b{B}_ctx{T}_ms_tok"] = round(per * 1e3, 3)
            out[f"decode_b{B}_ctx{T}_tok_s"] = round(B / per)
            clear_graph_cache()
    del model
    torch.cuda.empty_cache()
    return out


def run(sizes: List[str] = SIZES["vufilorn"], what=("prefill", "decode"), peer: bool = True) -> None:
    for name in sizes:
        cfg = get_config(name)
        rec = {"size": name, "layer_runs": len(cfg.layer_schedule), "width": cfg.hidden_size, "dtype": "bf16",
               "data": "synthetic", "model": measure(cfg, what)}
        if peer:
            for key, pc in peers(cfg).items():
                rec[key] = {"model": pc.name, "layers": pc.num_layers, "ff": pc.intermediate_size, **measure(pc, what)}
        print(json.dumps(rec), flush=True)
