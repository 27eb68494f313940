"""Model configurations + named presets (SURVEY Appendix B shapes).

The reference loads HF checkpoints by name (src/models/base_model.py:17-42). With no network,
the framework resolves `model_name_or_path` as: a local directory with config.json (HF layout,
loaded from safetensors), else a preset name below (random init), else a known HF hub id mapped
to its preset (e.g. "mistralai/Mistral-7B-v0.1" -> "mistral-7b", random init, shapes identical).
"""
from __future__ import annotations

import dataclasses
import json
from dataclasses import dataclass, field
from pathlib import Path
from typing import Any, Dict, List, Optional, Tuple


@dataclass
class ModelConfig:
    arch: str = "llama"  # llama | mistral | mixtral | gpt2 | phi | vufilorn | zenevik
    vocab_size: int = 32000
    hidden_size: int = 4096
    num_layers: int = 32
    num_heads: int = 32
    num_kv_heads: int = 8
    head_dim: int = 128
    intermediate_size: int = 14336
    norm_eps: float = 1e-5
    rope_theta: float = 10000.0
    rope_scaling: Optional[Dict[str, Any]] = None
    rotary_pct: float = 1.0
    max_position_embeddings: int = 8192
    sliding_window: int = 0
    tie_word_embeddings: bool = False
    num_experts: int = 0
    num_experts_per_tok: int = 2
    router_aux_loss_coef: float = 0.0
    norm_type: str = "rms"  # rms | layer
    activation: str = "swiglu"  # swiglu | geglu | gelu_new | relu2
    parallel_block: bool = False  # phi: attn and mlp both read the same normed input
    attn_bias: bool = False
    mlp_bias: bool = False
    lm_head_bias: bool = False
    learned_pos_emb: bool = False  # gpt2 wpe
    bos_token_id: int = 1
    eos_token_id: int = 2
    pad_token_id: Optional[int] = None
    init_std: float = 0.02
    name: str = "custom"
    # per-layer designs (models/mixers.py): one {"type", "mixer", "mlp"} dict per layer, each with
    # its own sizes; None = num_layers equal DecoderLayers described by the fields above
    layer_specs: Optional[List[Dict[str, Any]]] = None
    loop: Optional[Dict[str, int]] = None  # layers start .. stop-1 run `times` times in a row
    embed_scale: float = 1.0
    norm_offset: float = 0.0  # added to the stored norm weights (1.0: weights stored around zero)
    token_side_dim: int = 0  # per-layer token input: width of each layer's slice of side_embed
    postln_alpha: Optional[float] = None  # norm after the sum, x <- norm(alpha x + sublayer(x)); None: norm before
    logit_softcap: float = 0.0  # logits <- cap tanh(logits / cap)

    @property
    def layer_schedule(self) -> List[Tuple[int, bool]]:
        """The layer runs of one forward in order: (layer index, whether the embedding output is
        added to the stream first). Every run has its own cache / state slot."""
        n = self.num_layers
        if not self.loop:
            return [(i, False) for i in range(n)]
        a, b, times = int(self.loop["start"]), int(self.loop["stop"]), int(self.loop["times"])
        if not (0 <= a < b <= n and times >= 1):
            raise ValueError(f"loop {self.loop} does not fit {n} layers")
        runs = [(i, False) for i in range(a)]
        for p in range(times):
            runs += [(i, p > 0 and i == a) for i in range(a, b)]
        return runs + [(i, False) for i in range(b, n)]

    @property
    def q_size(self) -> int:
        return self.num_heads * self.head_dim

    @property
    def kv_size(self) -> int:
        return self.num_kv_heads * self.head_dim

    @property
    def rot_dim(self) -> int:
        if self.learned_pos_emb:
            return 0
        return int(self.head_dim * self.rotary_pct)

    @property
    def is_moe(self) -> bool:
        return self.num_experts > 0

    def num_params(self, include_embedding: bool = True) -> int:
        if self.layer_specs is not None:
            from .layer_spec import spec_param_count

            H, L, V = self.hidden_size, self.num_layers, self.vocab_size
            n = H + sum(spec_param_count(self, i) for i in range(L)) + (0 if self.tie_word_embeddings else V * H)
            return n + (V * H + V * L * self.token_side_dim if include_embedding else 0)
        H, F, L = self.hidden_size, self.intermediate_size, self.num_layers
        attn = H * (self.q_size + 2 * self.kv_size) + self.q_size * H
        mlp_one = (3 if self.activation == "swiglu" else 2) * H * F
        mlp = mlp_one * max(1, self.num_experts) + (H * self.num_experts if self.is_moe else 0)
        norms = (2 if not self.parallel_block else 1) * H
        per_layer = attn + mlp + norms
        emb = self.vocab_size * H if include_embedding else 0
        head = 0 if self.tie_word_embeddings else self.vocab_size * H
        return L * per_layer + emb + head + H

    def flops_per_token(self, seq_len: int) -> float:
        """Forward FLOPs/token: 2*matmul params (active experts only) + causal attention."""
        if self.layer_specs is not None:
            from .layer_spec import spec_flops_per_token

            return (2.0 * self.vocab_size * self.hidden_size
                    + sum(spec_flops_per_token(self, i, seq_len) for i, _ in self.layer_schedule))
        H, F, L = self.hidden_size, self.intermediate_size, self.num_layers
        attn_proj = H * (self.q_size + 2 * self.kv_size) + self.q_size * H
        n_mlp = self.num_experts_per_tok if self.is_moe else 1
        mlp = (3 if self.activation == "swiglu" else 2) * H * F * n_mlp
        matmul = L * (attn_proj + mlp) + self.vocab_size * H
        attn_scores = L * 2 * 2 * self.q_size * seq_len / 2  # QK^T + PV, causal half
        return 2.0 * matmul + attn_scores

    def to_dict(self) -> Dict[str, Any]:
        return dataclasses.asdict(self)

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "ModelConfig":
        names = {f.name for f in dataclasses.fields(cls)}
        return cls(**{k: v for k, v in d.items() if k in names})

    # ----------------------------------------------------------------- HF config.json interop
    @classmethod
    def from_hf(cls, hf: Dict[str, Any]) -> "ModelConfig":
        if "architecture" in hf:
            readers = {"Vufilorn": cls._from_vufilorn, "Zenevik": cls._from_zenevik}
            if hf["architecture"] not in readers:
                raise ValueError(f"unsupported architecture {hf['architecture']!r} (have {sorted(readers)})")
            return readers[hf["architecture"]](hf)
        mt = hf.get("model_type", "llama")
        if mt in ("llama", "mistral", "mixtral", "qwen2"):
            H = hf["hidden_size"]
            nh = hf["num_attention_heads"]
            return cls(
                arch=mt if mt != "qwen2" else "llama", vocab_size=hf["vocab_size"], hidden_size=H,
                num_layers=hf["num_hidden_layers"], num_heads=nh,
                num_kv_heads=hf.get("num_key_value_heads", nh),
                head_dim=hf.get("head_dim") or H // nh,
                intermediate_size=hf["intermediate_size"], norm_eps=hf.get("rms_norm_eps", 1e-6),
                rope_theta=hf.get("rope_theta", 10000.0), rope_scaling=hf.get("rope_scaling"),
                max_position_embeddings=hf.get("max_position_embeddings", 4096),
                sliding_window=hf.get("sliding_window") or 0,
                tie_word_embeddings=hf.get("tie_word_embeddings", False),
                num_experts=hf.get("num_local_experts", 0) if mt == "mixtral" else 0,
                num_experts_per_tok=hf.get("num_experts_per_tok", 2),
                router_aux_loss_coef=hf.get("router_aux_loss_coef", 0.0),
                attn_bias=hf.get("attention_bias", mt == "qwen2"),
                bos_token_id=hf.get("bos_token_id", 1) or 1, eos_token_id=_first(hf.get("eos_token_id", 2)),
                pad_token_id=hf.get("pad_token_id"), name=hf.get("_name_or_path", mt),
            )
        if mt == "gpt2":
            H = hf["n_embd"]
            nh = hf["n_head"]
            return cls(
                arch="gpt2", vocab_size=hf["vocab_size"], hidden_size=H, num_layers=hf["n_layer"],
                num_heads=nh, num_kv_heads=nh, head_dim=H // nh,
                intermediate_size=hf.get("n_inner") or 4 * H, norm_eps=hf.get("layer_norm_epsilon", 1e-5),
                max_position_embeddings=hf.get("n_positions", 1024), tie_word_embeddings=True,
                norm_type="layer", activation="gelu_new", attn_bias=True, mlp_bias=True,
                learned_pos_emb=True, bos_token_id=hf.get("bos_token_id", 50256),
                eos_token_id=hf.get("eos_token_id", 50256), name="gpt2",
            )
        if mt == "phi":
            H = hf["hidden_size"]
            nh = hf["num_attention_heads"]
            return cls(
                arch="phi", vocab_size=hf["vocab_size"], hidden_size=H,
                num_layers=hf["num_hidden_layers"], num_heads=nh,
                num_kv_heads=hf.get("num_key_value_heads") or nh, head_dim=H // nh,
                intermediate_size=hf["intermediate_size"], norm_eps=hf.get("layer_norm_eps", 1e-5),
                rope_theta=hf.get("rope_theta", 10000.0), rotary_pct=hf.get("partial_rotary_factor", 0.5),
                max_position_embeddings=hf.get("max_position_embeddings", 2048),
                norm_type="layer", activation="gelu_new", parallel_block=True, attn_bias=True,
                mlp_bias=True, lm_head_bias=True, bos_token_id=hf.get("bos_token_id", 50256) or 50256,
                eos_token_id=hf.get("eos_token_id", 50256) or 50256, name="phi",
            )
        raise ValueError(f"unsupported model_type {mt!r}")

    @classmethod
    def _from_vufilorn(cls, d: Dict[str, Any]) -> "ModelConfig":
        """Vufilorn config.json: `layers` lists each layer's mixer (latent attention or retention)
        and feed-forward with their own sizes; the flat head / FFN fields get the largest of them
        (reporting only, the layers read their specs)."""
        from .layer_spec import checked_specs

        specs = checked_specs(d["layers"], ("latent_attention", "retention"))
        mix = [e["mixer"] for e in specs]
        return cls(
            arch="vufilorn", vocab_size=d["vocab"], hidden_size=d["width"], num_layers=len(specs),
            num_heads=max(m["heads"] for m in mix), num_kv_heads=max(m["heads"] for m in mix),
            head_dim=max(m["dim"] + m.get("rot_dim", 0) for m in mix),
            intermediate_size=max([e["mlp"]["ff"] for e in specs if e.get("mlp")], default=0),
            norm_eps=d["norm"]["eps"], norm_offset=1.0, activation="relu2", tie_word_embeddings=True,
            max_position_embeddings=d.get("max_position_embeddings", 131072),
            layer_specs=specs, loop=d.get("loop"), embed_scale=float((d.get("embedding") or {}).get("scale", 1.0)),
            token_side_dim=int((d.get("token_side") or {}).get("dim", 0)),
            # the design names no special tokens: -1 = never sampled, generation runs to its length
            bos_token_id=d.get("bos_token_id", -1), eos_token_id=d.get("eos_token_id", -1), name="vufilorn")

    def _to_vufilorn(self) -> Dict[str, Any]:
        d = {"architecture": "Vufilorn", "vocab": self.vocab_size, "width": self.hidden_size,
             "embedding": {"scale": self.embed_scale}, "norm": {"eps": self.norm_eps},
             "layers": [dict(e) for e in self.layer_specs], "loop": self.loop,
             "token_side": {"dim": self.token_side_dim} if self.token_side_dim else None}
        for k in ("bos_token_id", "eos_token_id"):
            if getattr(self, k) >= 0:
                d[k] = getattr(self, k)
        return d

    @classmethod
    def _from_zenevik(cls, d: Dict[str, Any]) -> "ModelConfig":
        """Zenevik config.json: `layers` lists each layer's mixer (rglru, gla or attention in chunks)
        and optional feed-forward; norms come after the sums, and the logits are soft-capped."""
        from .layer_spec import checked_specs

        specs = checked_specs(d["layers"], ("rglru", "gla", "attention"))
        mix = [e["mixer"] for e in specs]
        return cls(
            arch="zenevik", vocab_size=d["vocab"], hidden_size=d["width"], num_layers=len(specs),
            num_heads=max(m.get("heads", 1) for m in mix),
            num_kv_heads=max(m.get("kv_heads", m.get("heads", 1)) for m in mix),
            head_dim=max(m.get("dim", 1) for m in mix),
            intermediate_size=max([e["mlp"]["ff"] for e in specs if e.get("mlp")], default=0),
            norm_eps=d["norm"]["eps"], activation="geglu", tie_word_embeddings=False,
            max_position_embeddings=d.get("max_position_embeddings", 131072), layer_specs=specs,
            postln_alpha=float(d["postln_alpha"]), logit_softcap=float(d["logit_softcap"]),
            # the design names no special tokens: -1 = never sampled, generation runs to its length
            bos_token_id=d.get("bos_token_id", -1), eos_token_id=d.get("eos_token_id", -1), name="zenevik")

    def _to_zenevik(self) -> Dict[str, Any]:
        d = {"architecture": "Zenevik", "vocab": self.vocab_size, "width": self.hidden_size,
             "norm": {"eps": self.norm_eps}, "postln_alpha": self.postln_alpha, "logit_softcap": self.logit_softcap,
             "layers": [dict(e) for e in self.layer_specs]}
        for k in ("bos_token_id", "eos_token_id"):
            if getattr(self, k) >= 0:
                d[k] = getattr(self, k)
        return d

    def to_hf(self) -> Dict[str, Any]:
        if self.arch == "vufilorn":
            return self._to_vufilorn()
        if self.arch == "zenevik":
            return self._to_zenevik()
        if self.arch == "gpt2":
            return {"model_type": "gpt2", "architectures": ["GPT2LMHeadModel"], "vocab_size": self.vocab_size,
                    "n_embd": self.hidden_size, "n_layer": self.num_layers, "n_head": self.num_heads,
                    "n_inner": self.intermediate_size, "n_positions": self.max_position_embeddings,
                    "layer_norm_epsilon": self.norm_eps, "activation_function": "gelu_new",
                    "bos_token_id": self.bos_token_id, "eos_token_id": self.eos_token_id,
                    "tie_word_embeddings": True, "torch_dtype": "bfloat16"}
        if self.arch == "phi":
            return {"model_type": "phi", "architectures": ["PhiForCausalLM"], "vocab_size": self.vocab_size,
                    "hidden_size": self.hidden_size, "num_hidden_layers": self.num_layers,
                    "num_attention_heads": self.num_heads, "num_key_value_heads": self.num_kv_heads,
                    "intermediate_size": self.intermediate_size, "layer_norm_eps": self.norm_eps,
                    "rope_theta": self.rope_theta, "partial_rotary_factor": self.rotary_pct,
                    "max_position_embeddings": self.max_position_embeddings, "hidden_act": "gelu_new",
                    "bos_token_id": self.bos_token_id, "eos_token_id": self.eos_token_id,
                    "torch_dtype": "bfloat16"}
        mt = self.arch
        arch_name = {"llama": "LlamaForCausalLM", "mistral": "MistralForCausalLM",
                     "mixtral": "MixtralForCausalLM"}[mt]
        d = {"model_type": mt, "architectures": [arch_name], "vocab_size": self.vocab_size,
             "hidden_size": self.hidden_size, "num_hidden_layers": self.num_layers,
             "num_attention_heads": self.num_heads, "num_key_value_heads": self.num_kv_heads,
             "head_dim": self.head_dim, "intermediate_size": self.intermediate_size,
             "rms_norm_eps": self.norm_eps, "rope_theta": self.rope_theta,
             "rope_scaling": self.rope_scaling, "max_position_embeddings": self.max_position_embeddings,
             "tie_word_embeddings": self.tie_word_embeddings, "hidden_act": "silu",
             "bos_token_id": self.bos_token_id, "eos_token_id": self.eos_token_id,
             "attention_bias": self.attn_bias, "torch_dtype": "bfloat16"}
        if mt in ("mistral", "mixtral"):
            d["sliding_window"] = self.sliding_window or None
        if mt == "mixtral":
            d["num_local_experts"] = self.num_experts
            d["num_experts_per_tok"] = self.num_experts_per_tok
            d["router_aux_loss_coef"] = self.router_aux_loss_coef
        return d


def _first(x):
    return x[0] if isinstance(x, (list, tuple)) else x


def _vufilorn_preset(vocab, width, order, ff, latent, retention, side_dim, scale, loop=None, eps=1e-6):
    """PRESETS entry of a Vufilorn model: `order` is one letter per layer, L(atent attention) or
    R(etention), all layers of a kind with the same sizes."""
    lat = {"type": "latent_attention", "mixer": latent, "mlp": {"kind": "dense", "ff": ff}}
    ret = {"type": "retention", "mixer": retention, "mlp": {"kind": "dense", "ff": ff}}
    return ModelConfig._from_vufilorn({
        "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps}, "loop": loop,
        "token_side": {"dim": side_dim}, "layers": [lat if c == "L" else ret for c in order]}).to_dict()


def _zenevik_preset(vocab, width, order, ff, lru, gla, attn, alpha, cap=30.0, eps=1e-6):
    """PRESETS entry of a Zenevik model: `order` is one letter per layer, R(ecurrent), G(ated linear
    attention) or A(ttention in chunks), all layers of a kind with the same sizes."""
    kinds = {"R": ("rglru", lru), "G": ("gla", gla), "A": ("attention", attn)}
    return ModelConfig._from_zenevik({
        "vocab": vocab, "width": width, "norm": {"eps": eps}, "postln_alpha": alpha, "logit_softcap": cap,
        "layers": [{"type": kinds[c][0], "mixer": kinds[c][1], "mlp": {"kind": "dense", "ff": ff}} for c in order]}).to_dict()


def _decays(heads: int, lo: float = 1 / 32, hi: float = 1 / 512) -> List[float]:
    """`heads` decays 1 - x, x log-spaced from lo to hi."""
    return [1.0 - lo * (hi / lo) ** (h / max(1, heads - 1)) for h in range(heads)]


PRESETS: Dict[str, Dict[str, Any]] = {
    # north-star models
    "llama3-8b": dict(arch="llama", vocab_size=128256, hidden_size=4096, num_layers=32, num_heads=32,
                      num_kv_heads=8, head_dim=128, intermediate_size=14336, norm_eps=1e-5,
                      rope_theta=500000.0, max_position_embeddings=8192, bos_token_id=128000,
                      eos_token_id=128001),
    "llama3-70b": dict(arch="llama", vocab_size=128256, hidden_size=8192, num_layers=80, num_heads=64,
                       num_kv_heads=8, head_dim=128, intermediate_size=28672, norm_eps=1e-5,
                       rope_theta=500000.0, max_position_embeddings=8192, bos_token_id=128000,
                       eos_token_id=128001),
    "mistral-7b": dict(arch="mistral", vocab_size=32000, hidden_size=4096, num_layers=32, num_heads=32,
                       num_kv_heads=8, head_dim=128, intermediate_size=14336, norm_eps=1e-5,
                       rope_theta=10000.0, max_position_embeddings=32768, sliding_window=4096),
    "mixtral-8x7b": dict(arch="mixtral", vocab_size=32000, hidden_size=4096, num_layers=32, num_heads=32,
                         num_kv_heads=8, head_dim=128, intermediate_size=14336, norm_eps=1e-5,
                         rope_theta=1e6, max_position_embeddings=32768, num_experts=8,
                         num_experts_per_tok=2, router_aux_loss_coef=0.02),
    "gpt2": dict(arch="gpt2", vocab_size=50257, hidden_size=768, num_layers=12, num_heads=12,
                 num_kv_heads=12, head_dim=64, intermediate_size=3072, norm_eps=1e-5,
                 max_position_embeddings=1024, tie_word_embeddings=True, norm_type="layer",
                 activation="gelu_new", attn_bias=True, mlp_bias=True, learned_pos_emb=True,
                 bos_token_id=50256, eos_token_id=50256),
    "phi-2": dict(arch="phi", vocab_size=51200, hidden_size=2560, num_layers=32, num_heads=32,
                  num_kv_heads=32, head_dim=80, intermediate_size=10240, norm_eps=1e-5,
                  rope_theta=10000.0, rotary_pct=0.4, max_position_embeddings=2048,
                  norm_type="layer", activation="gelu_new", parallel_block=True, attn_bias=True,
                  mlp_bias=True, lm_head_bias=True, bos_token_id=50256, eos_token_id=50256),
    # test-scale models (CPU tier / smoke)
    "tiny-llama": dict(arch="llama", vocab_size=512, hidden_size=128, num_layers=2, num_heads=4,
                       num_kv_heads=2, head_dim=32, intermediate_size=256, norm_eps=1e-5,
                       rope_theta=10000.0, max_position_embeddings=512, bos_token_id=1, eos_token_id=2),
    "tiny-llama-d128": dict(arch="llama", vocab_size=1024, hidden_size=512, num_layers=2, num_heads=4,
                            num_kv_heads=2, head_dim=128, intermediate_size=1024, norm_eps=1e-5,
                            rope_theta=500000.0, max_position_embeddings=2048, bos_token_id=1,
                            eos_token_id=2),
    "tiny-mistral": dict(arch="mistral", vocab_size=512, hidden_size=128, num_layers=2, num_heads=4,
                         num_kv_heads=2, head_dim=32, intermediate_size=256, norm_eps=1e-5,
                         max_position_embeddings=512, sliding_window=16),
    "tiny-mixtral": dict(arch="mixtral", vocab_size=512, hidden_size=128, num_layers=2, num_heads=4,
                         num_kv_heads=2, head_dim=32, intermediate_size=128, norm_eps=1e-5,
                         max_position_embeddings=512, num_experts=4, num_experts_per_tok=2),
    "tiny-gpt2": dict(arch="gpt2", vocab_size=512, hidden_size=128, num_layers=2, num_heads=4,
                      num_kv_heads=4, head_dim=32, intermediate_size=512, max_position_embeddings=512,
                      tie_word_embeddings=True, norm_type="layer", activation="gelu_new",
                      attn_bias=True, mlp_bias=True, learned_pos_emb=True, bos_token_id=1,
                      eos_token_id=2),
    "tiny-phi": dict(arch="phi", vocab_size=512, hidden_size=160, num_layers=2, num_heads=2,
                     num_kv_heads=2, head_dim=80, intermediate_size=320, rotary_pct=0.4,
                     max_position_embeddings=512, norm_type="layer", activation="gelu_new",
                     parallel_block=True, attn_bias=True, mlp_bias=True, lm_head_bias=True,
                     bos_token_id=1, eos_token_id=2),
}

PRESETS.update({
    # Vufilorn (latent attention in a window + retention, looped layers, per-layer token input)
    "tiny-vufilorn": _vufilorn_preset(
        320, 96, "RLL", 160,
        dict(heads=3, dim=16, rot_dim=8, vdim=24, kv_rank=40, q_rank=32, scale=0.2,
             rot=dict(base=10000.0, dims=8), mask=dict(size=11)),
        dict(heads=2, dim=24, vdim=40, rot=dict(base=500.0, dims=16), decay=[0.9, 0.97]),
        side_dim=8, scale=3.0, loop=dict(start=1, stop=3, times=2)),
    "vufilorn-1b": _vufilorn_preset(
        32000, 2048, "LRLRLRLRLRLR", 8192,
        dict(heads=16, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=768, scale=192 ** -0.5,
             rot=dict(base=1e6, dims=64), mask=dict(size=4096)),
        dict(heads=16, dim=128, vdim=128, rot=dict(base=1e6, dims=128), decay=_decays(16)),
        side_dim=128, scale=45.0, loop=dict(start=2, stop=10, times=2)),
    "vufilorn-7b": _vufilorn_preset(
        32000, 4096, "LRLRLRLRLRLRLRLRLRLR", 16384,
        dict(heads=32, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=1536, scale=192 ** -0.5,
             rot=dict(base=1e6, dims=64), mask=dict(size=4096)),
        dict(heads=16, dim=256, vdim=256, rot=dict(base=1e6, dims=256), decay=_decays(16)),
        side_dim=256, scale=64.0, loop=dict(start=4, stop=16, times=2)),
})

PRESETS.update({
    # Zenevik (real-gated recurrence, gated linear attention, attention in chunks; norm after the sum)
    "tiny-zenevik": _zenevik_preset(
        320, 96, "RGAR", 160, dict(width=128, blocks=4, conv=4),
        dict(heads=3, dim=16, vdim=24, tau=8.0, rank=16),
        dict(heads=4, kv_heads=2, dim=24, vdim=24, scale=0.2, rot=dict(base=10000.0, dims=16), mask=dict(size=11)), 2.0),
    "zenevik-1b": _zenevik_preset(
        32000, 2048, "RGARGARGARGARGAR", 5632, dict(width=2560, blocks=10, conv=4),
        dict(heads=16, dim=128, vdim=128, tau=16.0, rank=16),
        dict(heads=16, kv_heads=4, dim=128, vdim=128, scale=128 ** -0.5, rot=dict(base=1e6, dims=64),
             mask=dict(size=4096)), 3.0),
    "zenevik-7b": _zenevik_preset(
        32000, 4096, "RGARGARGARGARGARGARGARGARGARGARG", 11264, dict(width=4096, blocks=16, conv=4),
        dict(heads=16, dim=128, vdim=256, tau=16.0, rank=16),
        dict(heads=32, kv_heads=8, dim=128, vdim=128, scale=128 ** -0.5, rot=dict(base=1e6, dims=64),
             mask=dict(size=4096)), 3.0),
})

# HF hub ids used by the reference configs -> presets (random init offline, identical shapes)
HUB_ALIASES = {
    "mistralai/Mistral-7B-v0.1": "mistral-7b",
    "meta-llama/Meta-Llama-3-8B": "llama3-8b",
    "meta-llama/Meta-Llama-3-8B-Instruct": "llama3-8b",
    "meta-llama/Meta-Llama-3-70B": "llama3-70b",
    "mistralai/Mixtral-8x7B-v0.1": "mixtral-8x7b",
    "microsoft/phi-2": "phi-2",
    "gpt2": "gpt2",
    "openai-community/gpt2": "gpt2",
}


def tp_shard_config(cfg: ModelConfig, tp: int) -> ModelConfig:
    """The per-rank shapes of `cfg` under tensor parallelism of degree `tp` as a standalone
    (world-1) model: heads, KV heads, FFN width and vocabulary divided by tp, hidden size and
    depth kept. Used by `bench.py --tp-shape` to time one TP rank's real GEMM / attention / norm
    shapes on one GPU (e.g. Llama-3-70B at tp 8: 8 q heads / 1 kv head, FFN 3584, vocab 16032)."""
    if cfg.layer_specs is not None:
        raise ValueError(f"{cfg.name}: per-layer designs have no tensor-parallel form")
    if cfg.num_heads % tp or cfg.num_kv_heads % tp or cfg.intermediate_size % tp or cfg.vocab_size % tp:
        raise ValueError(f"{cfg.name}: heads / kv heads / FFN / vocab must divide tp={tp}")
    d = cfg.to_dict()
    d.update(num_heads=cfg.num_heads // tp, num_kv_heads=cfg.num_kv_heads // tp,
             intermediate_size=cfg.intermediate_size // tp, vocab_size=cfg.vocab_size // tp,
             name=f"{cfg.name}@tp{tp}")
    return ModelConfig.from_dict(d)


def _with_tensor_sizes(hf: Dict[str, Any], path: Path) -> Dict[str, Any]:
    """Fill in the sizes that a per-layer design's config.json leaves to its tensors' shapes."""
    from .layer_spec import TENSOR_SIZES

    layers = hf.get("layers") if "architecture" in hf else None
    open_sizes = [(e["mixer"], f"l{i}.{tensor}", axis, key) for i, e in enumerate(layers or [])
                  for key, tensor, axis in TENSOR_SIZES.get(e.get("type"), ()) if key not in e["mixer"]]
    if open_sizes:
        from .loader import read_state_dict

        sd = read_state_dict(path)
        for mixer, tensor, axis, key in open_sizes:
            if tensor in sd:
                mixer[key] = int(sd[tensor].shape[axis])
    return hf


def get_config(name_or_path: str, **overrides) -> ModelConfig:
    """Resolve a preset / HF directory / hub alias into a ModelConfig. `<preset>@tp<N>` gives the
    per-rank shard shapes of that preset under TP degree N (tp_shard_config)."""
    name = str(name_or_path)
    if "@tp" in name and not Path(name).is_dir():
        base, tp = name.rsplit("@tp", 1)
        cfg = tp_shard_config(get_config(base), int(tp))
        for k, v in overrides.items():
            setattr(cfg, k, v)
        return cfg
    p = Path(str(name_or_path))
    if p.is_dir():
        if (p / "dla_config.json").exists():
            cfg = ModelConfig.from_dict(json.loads((p / "dla_config.json").read_text()))
        elif (p / "config.json").exists():
            cfg = ModelConfig.from_hf(_with_tensor_sizes(json.loads((p / "config.json").read_text()), p))
        else:
            raise FileNotFoundError(f"{p} has no config.json")
    else:
        key = HUB_ALIASES.get(str(name_or_path), str(name_or_path))
        if key not in PRESETS:
            raise KeyError(f"unknown model {name_or_path!r}; presets: {sorted(PRESETS)}")
        cfg = ModelConfig(**{**PRESETS[key], "name": key})
    for k, v in overrides.items():
        setattr(cfg, k, v)
    return cfg
