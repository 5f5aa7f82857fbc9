"""Workload shapes of the fused LoRA SFT step (the five benchmark configurations).

Field names follow the reference's SFTState dims (src/nn/fast_sft.c:33-44):
NL layers, D hidden, Hq/Hkv heads, hd head dim, IS FFN width, V vocab.
"""
from dataclasses import dataclass, replace

QWEN3, GEMMA3, NEVURAX, PAPOSUN = 0, 1, 2, 3     # ModelType of include/sft_hip.h


@dataclass(frozen=True)
class SFTConfig:
    name: str
    model_type: int          # QWEN3 | GEMMA3
    NL: int
    D: int
    Hq: int
    Hkv: int
    hd: int
    IS: int
    V: int
    batch: int = 1
    seq: int = 64
    R: int = 16              # LoRA rank
    alpha: float = 32.0
    eps: float = 1e-6        # src/nn/fast_sft.c:190
    rope_theta: float = 1e6  # Qwen3: every layer; Gemma3: global layers (L % 6 == 0)
    local_rope_theta: float = 1e4   # Gemma3 local layers (src/nn/fast_sft.c:310-313)
    tied: bool = False       # lm_head shares the embedding table
    weight_format: str = "f16"      # "f16" | "q8_0"
    window: int = 0          # sliding-window attention on the local layers (0 = off: the reference never applies it)

    @property
    def BN(self):
        return self.batch * self.seq

    @property
    def lora_scaling(self):
        return self.alpha / self.R

    @property
    def emb_scale(self):
        import numpy as np
        return float(np.sqrt(np.float32(self.D))) if self.model_type == GEMMA3 else 1.0

    def rope_thetas(self):
        if self.model_type == GEMMA3:
            return [self.rope_theta if (L % 6) == 0 else self.local_rope_theta for L in range(self.NL)]
        return [self.rope_theta] * self.NL

    def local_layers(self):
        """Layers the sliding window applies to: Gemma3's pattern (src/nn/gemma3.c:49-57), every layer otherwise."""
        return [(L % 6) != 0 if self.model_type == GEMMA3 else True for L in range(self.NL)]

    @property
    def lora_layer_size(self):
        return 2 * self.R * self.D + self.Hq * self.hd * self.R + self.Hkv * self.hd * self.R

    @property
    def frozen_params(self):
        per = (self.Hq * self.hd + 2 * self.Hkv * self.hd) * self.D + self.D * self.Hq * self.hd + 3 * self.IS * self.D
        return per * self.NL + self.V * self.D

    def with_(self, **kw):
        return replace(self, **kw)


C1 = SFTConfig("c1_tiny_qwen3", QWEN3, NL=2, D=256, Hq=4, Hkv=2, hd=64, IS=768, V=4096, tied=True)
C2 = SFTConfig("c2_gemma3_1b", GEMMA3, NL=26, D=1152, Hq=4, Hkv=1, hd=256, IS=6912, V=262144, tied=True)
C3 = SFTConfig("c3_qwen3_4b_f16", QWEN3, NL=36, D=2560, Hq=32, Hkv=8, hd=128, IS=9728, V=151936)
C4 = C3.with_(name="c4_qwen3_4b_q8", batch=4, seq=512, weight_format="q8_0")
# the group of four 160-token sequences is one batch: a pass streams every weight once for the whole group
C5 = C2.with_(name="c5_gemma3_1b_grpo", batch=4, seq=160, R=0)
# config 3's step on Q8_0 weights: the dequant-fused weight-streaming GEMM at M = 64
C3Q = C3.with_(name="c3_qwen3_4b_q8_seq64", weight_format="q8_0")

# small Gemma3-shaped case for parity tests (4-norm ordering, GeGLU, tied head, mixed thetas)
TINY_GEMMA3 = SFTConfig("tiny_gemma3", GEMMA3, NL=7, D=128, Hq=4, Hkv=1, hd=32, IS=384, V=2048, tied=True, seq=32)

CONFIGS = {c.name: c for c in (C1, C2, C3, C4, C5, C3Q, TINY_GEMMA3)}


def nevurax_config(width, heads, ff, experts, top, shared_ff, vocab=32768, head_dim=128, rot_dim=64, kv_rank=512, window=1024,
                   order=("channel_delta", "latent_attention", "delta", "channel_delta")):
    """config.json of a Nevurax model with layers of a real model's proportions (one width of heads for all mixers)."""
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}, "shared": {"ff": shared_ff}}
    rule = {"heads": heads, "kv_heads": heads, "dim": head_dim, "vdim": head_dim, "conv": 4}
    latent = {"heads": heads, "dim": head_dim, "rot_dim": rot_dim, "vdim": head_dim, "kv_rank": kv_rank, "mask": {"size": window},
              "rot": {"base": 1e4, "dims": rot_dim}, "scale": (head_dim + rot_dim) ** -0.5}
    return {"architecture": "Nevurax", "vocab": vocab, "width": width, "embedding": {"scale": 1.0}, "norm": {"eps": 1e-6},
            "layers": [{"type": t, "mixer": latent if t == "latent_attention" else rule, "mlp": mlp} for t in order]}


# benchmark sizes: four layers each, beside a Qwen3-shaped model of the same width, heads and active FFN weights per token
NEVURAX_SIZES = {
    "1k": nevurax_config(1024, 8, 512, 32, 4, 1024),
    "2k": nevurax_config(2048, 16, 768, 64, 6, 1536),
    "4k": nevurax_config(4096, 32, 1024, 32, 8, 2048),
}


def paposun_config(width, heads, ff, memory_heads, memory_dim, vocab=32768, head_dim=128, chunk=1024):
    """config.json of a Paposun model with layers of a real model's proportions: attention, attention on the same keys, mLSTM
    (values twice as wide as keys, as wide together as the model), attention."""
    def attention(**kw):
        return {"type": "attention", "mlp": {"kind": "dense", "ff": ff},
                "mixer": {"heads": heads, "kv_heads": max(1, heads // 4), "dim": head_dim, "vdim": head_dim, "mask": {"size": chunk}, "scale": head_dim ** -0.5,
                          "rot": {"base": 1e6, "dims": head_dim, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}, **kw}}
    memory = {"type": "mlstm", "mlp": None, "mixer": {"heads": memory_heads, "dim": memory_dim, "vdim": 2 * memory_dim, "gate_cap": 15.0}}
    return {"architecture": "Paposun", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "residual_mult": 0.5, "logit_scale": 0.5,
            "layers": [attention(), attention(kv_from=0), memory, attention()]}


PAPOSUN_SIZES = {
    "1k": paposun_config(1024, 8, 4096, 4, 128),
    "2k": paposun_config(2048, 16, 8192, 4, 256),
    "4k": paposun_config(4096, 32, 16384, 8, 256),
}


def qwen3_beside(cfg):
    """The Qwen3 shape with a layer-by-layer configuration's width, layers, heads and feed-forward weights per token."""
    active = 0
    for L in cfg["layers"]:
        m = L["mlp"]
        if m:
            active += 2 * (m["ff"] if m["kind"] == "dense" else m["router"]["top"] * m["expert"]["ff"] + m["shared"]["ff"])
    NL, mx = len(cfg["layers"]), cfg["layers"][0]["mixer"]
    return SFTConfig("qwen3_beside_layered", QWEN3, NL=NL, D=cfg["width"], Hq=mx["heads"], Hkv=max(1, mx["heads"] // 4),
                     hd=mx["dim"], IS=active // NL // 3 // 64 * 64, V=cfg["vocab"])
