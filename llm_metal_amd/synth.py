"""Seeded synthetic models and batches for the SFT step.

Weights ~ N(0, 0.02), norm gammas = 1 (rms_norm_create, src/nn/layers.c:336-344),
LoRA A ~ U(-1, 1)/sqrt(D) (src/nn/fast_sft.c:100-104), B = 0 for timing runs or
N(0, 0.01) for parity runs (a zero B makes the first-step dA exactly zero),
tokens uniform on [0, V), target = next token with the last wrapping to the
first (main.c:471-477).
"""
import os

import numpy as np
from .configs import SFTConfig, GEMMA3

MATS = ("wq", "wk", "wv", "wo", "wg", "wu", "wd")


def mat_shapes(c: SFTConfig):
    qd, kd = c.Hq * c.hd, c.Hkv * c.hd
    return {"wq": (qd, c.D), "wk": (kd, c.D), "wv": (kd, c.D), "wo": (c.D, qd),
            "wg": (c.IS, c.D), "wu": (c.IS, c.D), "wd": (c.D, c.IS)}


def _normal(rng, shape, std):
    a = rng.standard_normal(shape, dtype=np.float32)
    a *= np.float32(std)
    return a


def make_model(c: SFTConfig, seed=0, gamma_jitter=0.0, lora_b_std=0.01, threads=None):
    """Returns a dict of fp32 numpy arrays: per-layer lists for the 7 matrices and
    the norm gammas, token_emb, lm_head (same object when tied), g_final, lora
    (flat [NL * lora_layer_size]: A_q | B_q | A_v | B_v per layer).  Every array has
    its own generator derived from (seed, index), so the result does not depend on
    how many threads filled it."""
    from concurrent.futures import ThreadPoolExecutor
    shp = mat_shapes(c)
    m = {k: [None] * c.NL for k in MATS}
    jobs = []                                              # (dict, key/index, shape)
    for L in range(c.NL):
        for k in MATS:
            jobs.append((m[k], L, shp[k]))
    m["token_emb"] = None
    jobs.append((m, "token_emb", (c.V, c.D)))
    if not c.tied:
        jobs.append((m, "lm_head", (c.V, c.D)))
    seqs = np.random.SeedSequence(seed).spawn(len(jobs) + 2)

    def fill(i):
        dst, key, shape = jobs[i]
        dst[key] = _normal(np.random.default_rng(seqs[i]), shape, 0.02)

    big = sum(int(np.prod(j[2])) for j in jobs) > 50_000_000
    if big:
        with ThreadPoolExecutor(threads or min(16, (os.cpu_count() or 8))) as ex:
            list(ex.map(fill, range(len(jobs))))
    else:
        for i in range(len(jobs)):
            fill(i)
    if c.tied:
        m["lm_head"] = m["token_emb"]

    rng = np.random.default_rng(seqs[-2])

    def gamma(n):
        g = np.ones(n, dtype=np.float32)
        if gamma_jitter:
            g += _normal(rng, n, gamma_jitter)
        return g

    for k in ("g_in", "g_post_attn", "g_pre_ff", "g_post_ff", "g_q", "g_k"):
        m[k] = []
    for _ in range(c.NL):
        m["g_in"].append(gamma(c.D))
        m["g_post_attn"].append(gamma(c.D))
        m["g_pre_ff"].append(gamma(c.D) if c.model_type == GEMMA3 else None)
        m["g_post_ff"].append(gamma(c.D) if c.model_type == GEMMA3 else None)
        m["g_q"].append(gamma(c.hd))
        m["g_k"].append(gamma(c.hd))
    m["g_final"] = gamma(c.D)
    m["lora"] = make_lora(c, np.random.default_rng(seqs[-1]), lora_b_std)
    return m


def make_lora(c: SFTConfig, rng, lora_b_std):
    if c.R == 0:
        return np.zeros(0, dtype=np.float32)
    qd, kd = c.Hq * c.hd, c.Hkv * c.hd
    parts = []
    for _ in range(c.NL):
        for rows, cols, is_a in ((c.R, c.D, True), (qd, c.R, False), (c.R, c.D, True), (kd, c.R, False)):
            if is_a:
                a = (rng.random((rows, cols), dtype=np.float32) * 2 - 1) / np.float32(np.sqrt(c.D))
            elif lora_b_std:
                a = _normal(rng, (rows, cols), lora_b_std)
            else:
                a = np.zeros((rows, cols), dtype=np.float32)
            parts.append(a.astype(np.float32).ravel())
    return np.concatenate(parts)


def lora_views(c: SFTConfig, flat):
    """Split a flat LoRA arena into per-layer dicts of (A_q, B_q, A_v, B_v) views."""
    qd, kd = c.Hq * c.hd, c.Hkv * c.hd
    out, o = [], 0
    for _ in range(c.NL):
        d = {}
        for name, (r, k) in (("A_q", (c.R, c.D)), ("B_q", (qd, c.R)), ("A_v", (c.R, c.D)), ("B_v", (kd, c.R))):
            d[name] = flat[o:o + r * k].reshape(r, k)
            o += r * k
        out.append(d)
    return out


def make_batch(c: SFTConfig, seed=1):
    rng = np.random.default_rng(seed)
    tok = rng.integers(0, c.V, size=(c.batch, c.seq), dtype=np.uint32)
    tgt = np.roll(tok, -1, axis=1)
    return tok.reshape(-1).copy(), tgt.reshape(-1).copy()


# ---------------------------------------------------------------- models described layer by layer (Nevurax, Paposun)

def stack_shapes(cfg, rank_a=16, rank_g=16):
    """Tensor names and shapes of a layer-by-layer model; cfg is the dictionary that becomes its config.json.  rank_a and
    rank_g: widths of the two low-rank products of a per-channel decay (tensor shapes, not configuration)."""
    if cfg["architecture"] == "Paposun":
        return around_shapes(cfg)
    D = cfg["width"]
    out = {"embed": (cfg["vocab"], D)}
    for i, L in enumerate(cfg["layers"]):
        m, p = L["mixer"], f"l{i}."
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        out[p + "norm1"] = (D,)
        x = p + "mix."
        if L["type"] == "latent_attention":
            r, R = m["rot_dim"], m["kv_rank"]
            out.update({x + "q": (H * (d + r), D), x + "dkv": (R + r, D), x + "dkv.norm": (R,), x + "uk": (H * d, R), x + "uv": (H * dv, R)})
        else:
            kd = m["kv_heads"] * d
            for n, c in (("q", kd), ("k", kd), ("v", H * dv)):
                out.update({x + n: (c, D), x + n + ".conv": (c, m["conv"])})
            out.update({x + "b": (H, D), x + "A_log": (H,), x + "norm": (dv,)})
            if L["type"] == "channel_delta":
                out.update({x + "a1": (rank_a, D), x + "a2": (H * d, rank_a), x + "dt_bias": (H * d,),
                            x + "g1": (rank_g, D), x + "g2": (H * dv, rank_g)})
            else:
                out.update({x + "a": (H, D), x + "dt_bias": (H,), x + "g": (H * dv, D)})
        out[x + "o"] = (D, H * dv)
        if L.get("mlp"):
            e, f, y = L["mlp"]["router"]["experts"], L["mlp"]["expert"]["ff"], p + "mlp."
            for k in range(e):
                out.update({f"{y}e{k}.up": (f, D), f"{y}e{k}.down": (D, f)})
            out[y + "router"] = (e, D)
            if L["mlp"].get("shared"):
                s = L["mlp"]["shared"]["ff"]
                out.update({y + "shared.up": (s, D), y + "shared.down": (D, s)})
    out.update({"final.norm": (D,), "head": (cfg["vocab"], D)})
    return out


def around_shapes(cfg):
    """The same for norms around the sublayers: grouped attention with biases, mLSTM, dense feed-forward, tied head."""
    D = cfg["width"]
    out = {"embed": (cfg["vocab"], D)}
    for i, L in enumerate(cfg["layers"]):
        m, p = L["mixer"], f"l{i}."
        H, d, dv, x = m["heads"], m["dim"], m["vdim"], p + "mix."
        out.update({p + "norm1": (D,), p + "norm1b": (D,)})

        def biased(name, rows):
            out.update({x + name: (rows, D), x + name + ".b": (rows,)})
        if L["type"] == "attention":
            biased("q", H * d)
            if m.get("kv_from") is None:
                biased("k", m["kv_heads"] * d)
                biased("v", m["kv_heads"] * dv)
            out.update({x + "g": (H * dv, D), x + "o": (D, H * dv), x + "o.b": (D,)})
        else:
            out.update({x + "q": (H * d, D), x + "k": (H * d, D), x + "v": (H * dv, D), x + "g": (H * dv, D), x + "o": (D, H * dv), x + "norm": (H * dv,)})
            biased("i", H)
            biased("f", H)
        if L.get("mlp"):
            out.update({p + "norm2": (D,), p + "norm2b": (D,), p + "mlp.up": (L["mlp"]["ff"], D), p + "mlp.down": (D, L["mlp"]["ff"])})
    out["final.norm"] = (D,)
    return out


def make_stack_tensor(name, shape, rng):
    """Matrices ~ N(0, 1 / columns) (down and output projections half of that), norms around 1, filters and decay
    parameters and gate biases spread so that states remember from a few tokens to a few hundred, other biases small."""
    leaf = name.rsplit(".", 1)[-1]
    if leaf in ("norm", "norm1", "norm1b", "norm2", "norm2b"):
        return (1.0 + 0.1 * rng.standard_normal(shape)).astype(np.float32)
    if leaf == "b" and len(shape) == 1:
        if name.endswith(".f.b"):
            return rng.uniform(1.0, 6.0, shape).astype(np.float32)
        return (0.3 * rng.standard_normal(shape)).astype(np.float32)
    if leaf == "conv":
        return (rng.standard_normal(shape) / np.sqrt(shape[1])).astype(np.float32)
    if leaf == "A_log":
        return rng.uniform(-3.0, 0.5, shape).astype(np.float32)
    if leaf == "dt_bias":
        return rng.uniform(-3.0, 0.0, shape).astype(np.float32)
    if leaf == "embed":
        return rng.standard_normal(shape, dtype=np.float32)
    scale = (0.5 if leaf in ("down", "o") else 1.0) / np.sqrt(shape[-1])
    a = rng.standard_normal(shape, dtype=np.float32)
    a *= np.float32(scale)
    return a


def to_bf16_bits(a):
    b = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((b + np.uint32(0x7FFF) + ((b >> np.uint32(16)) & np.uint32(1))) >> np.uint32(16)).astype(np.uint16)


def write_stack_checkpoint(path, cfg, seed=0, rank_a=16, rank_g=16, keep=False, edit=None, repeat=False):
    """config.json and model.safetensors (bfloat16) of a random model in the folder `path`.  keep: return the values the
    file holds, fp32 by name.  edit(name, array): may replace a tensor before it is rounded.  repeat: every matrix of the
    experts is the same one (large models for timing, written in a fraction of the time)."""
    import json
    import struct
    shapes = stack_shapes(cfg, rank_a, rank_g)
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, off = {}, 0
    for name, shape in shapes.items():
        n = 2 * int(np.prod(shape))
        header[name] = {"dtype": "BF16", "shape": list(shape), "data_offsets": [off, off + n]}
        off += n
    text = json.dumps(header).encode()
    text += b" " * (-len(text) % 8)
    kept, drawn = {}, {}
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(text)) + text)
        for i, (name, shape) in enumerate(shapes.items()):
            kind = (name.rsplit(".", 1)[-1], shape)
            if repeat and ".e" in name and kind in drawn:
                f.write(drawn[kind])
                continue
            a = make_stack_tensor(name, shape, np.random.default_rng([seed, i]))
            if edit is not None:
                a = edit(name, a)
            bits = to_bf16_bits(a)
            f.write(bits.tobytes())
            if repeat and ".e" in name:
                drawn[kind] = bits.tobytes()
            if keep:
                kept[name] = (bits.astype(np.uint32) << np.uint32(16)).view(np.float32)
    return kept
