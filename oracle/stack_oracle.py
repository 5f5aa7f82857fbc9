"""Plain restatement, in numpy and one token at a time, of decoders whose layers are listed one by one.

Nevurax: short causal convolutions, the gated delta rule with one decay per head or per key channel, latent attention with
a sliding window and interleaved rotation, squared-ReLU experts behind a softmax router, one layer norm per layer whose
output both sublayers read.  Paposun: grouped attention inside fixed chunks of positions with biases, half-split rotation
of scaled frequencies, an output gate and keys that later layers may share, the mLSTM matrix memory, a dense tanh-GELU
feed-forward, RMS norms before and after each sublayer.

Test infrastructure only: nothing here is used by the package, and nothing of the package is used here.  Everything runs in
the dtype of the weights handed in (float64 for pinning).  A model is a config dictionary (its config.json) and a
dictionary of numpy arrays by tensor name.
"""
import numpy as np


# ---------------------------------------------------------------- elementwise

def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def relu2(z):
    r = np.maximum(z, 0.0)
    return r * r


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


# ---------------------------------------------------------------- norms and rotation

def layer_norm(x, w, eps):
    d = x - x.mean()
    return d / np.sqrt((d * d).mean() + eps) * w


def rms_norm(x, w, eps):
    return x / np.sqrt((x * x).mean() + eps) * w


def unit(x):
    return x / np.sqrt((x * x).sum() + 1e-6)


def rotate_interleaved(x, pos, dims, base):
    """Pairs (2i, 2i + 1) of the first `dims` entries turned by pos * base^(-2i / dims)."""
    y = x.copy()
    for i in range(dims // 2):
        a = pos * float(base) ** (-2.0 * i / dims)
        c, s = np.cos(a), np.sin(a)
        u, v = x[2 * i], x[2 * i + 1]
        y[2 * i], y[2 * i + 1] = u * c - v * s, v * c + u * s
    return y


def scaled_frequencies(rot):
    """Angles per position of the pairs.  Wavelengths above original / low are stretched by `factor`, those below
    original / high are kept, a linear mix in between."""
    out, sc = [], rot.get("scaling")
    for i in range(rot["dims"] // 2):
        f = float(rot["base"]) ** (-2.0 * i / rot["dims"])
        if sc:
            turns = sc["original"] * f / (2.0 * np.pi)          # turns within the original context
            if turns < sc["low"]:
                f = f / sc["factor"]
            elif turns <= sc["high"]:
                mix = (turns - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - mix) * f / sc["factor"] + mix * f
        out.append(f)
    return out


def rotate_halves(x, pos, rot):
    """Entry i turned together with entry i + dims / 2, i < dims / 2."""
    y, n = x.copy(), rot["dims"] // 2
    for i, f in enumerate(scaled_frequencies(rot)):
        c, s = np.cos(pos * f), np.sin(pos * f)
        y[i], y[i + n] = x[i] * c - x[i + n] * s, x[i + n] * c + x[i] * s
    return y


# ---------------------------------------------------------------- mixers; `state` is a dictionary kept per sequence and layer

def short_conv(state, key, x, taps):
    """Causal convolution over time, one filter per channel; taps[:, -1] meets the current input."""
    n = taps.shape[1]
    past = state.setdefault(key, [np.zeros_like(x)] * (n - 1))
    window = past + [x]
    y = sum(window[i] * taps[:, i] for i in range(n))
    state[key] = window[1:] if n > 1 else []
    return y


def delta_step(S, q, k, v, g, beta):
    """One head, one token.  S [dim, vdim]; g scalar or [dim]."""
    S = (g[:, None] if np.ndim(g) else g) * S
    u = beta * (v - S.T @ k)
    S = S + np.outer(k, u)
    return S, S.T @ q


def delta_mixer(W, p, mx, eps, per_channel, state, h, pos):
    H, KV, d, dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = silu(short_conv(state, "q", W[p + "q"] @ h, W[p + "q.conv"])).reshape(KV, d)
    k = silu(short_conv(state, "k", W[p + "k"] @ h, W[p + "k.conv"])).reshape(KV, d)
    v = silu(short_conv(state, "v", W[p + "v"] @ h, W[p + "v.conv"])).reshape(H, dv)
    q = np.stack([unit(r) for r in q]) / np.sqrt(d)
    k = np.stack([unit(r) for r in k])
    beta = sigmoid(W[p + "b"] @ h)
    if per_channel:
        a = softplus(W[p + "a2"] @ (W[p + "a1"] @ h) + W[p + "dt_bias"]).reshape(H, d)
        g = np.exp(-np.exp(W[p + "A_log"])[:, None] * a)
        gate = sigmoid(W[p + "g2"] @ (W[p + "g1"] @ h)).reshape(H, dv)
    else:
        g = np.exp(-np.exp(W[p + "A_log"]) * softplus(W[p + "a"] @ h + W[p + "dt_bias"]))
        gate = silu(W[p + "g"] @ h).reshape(H, dv)
    S = state.setdefault("S", np.zeros((H, d, dv), dtype=h.dtype))
    out = np.zeros((H, dv), dtype=h.dtype)
    new = np.empty_like(S)
    for i in range(H):
        j = i // (H // KV)
        new[i], o = delta_step(S[i], q[j], k[j], v[i], g[i], beta[i])
        out[i] = rms_norm(o, W[p + "norm"], eps) * gate[i]
    state["S"] = new
    return W[p + "o"] @ out.reshape(-1)


def latent_attention(W, p, mx, eps, state, h, pos):
    H, d, r, dv, R = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
    rot, window, scale = mx["rot"], mx["mask"]["size"], mx["scale"]
    q = (W[p + "q"] @ h).reshape(H, d + r)
    dkv = W[p + "dkv"] @ h
    cs, ks = state.setdefault("c", []), state.setdefault("k", [])
    cs.append(rms_norm(dkv[:R], W[p + "dkv.norm"], eps))
    ks.append(rotate_interleaved(dkv[R:], pos, rot["dims"], rot["base"]))
    first = max(0, pos - window + 1)
    c, kr = np.stack(cs[first:pos + 1]), np.stack(ks[first:pos + 1])
    uk, uv = W[p + "uk"].reshape(H, d, R), W[p + "uv"].reshape(H, dv, R)
    out = np.zeros((H, dv), dtype=h.dtype)
    for i in range(H):
        qr = rotate_interleaved(q[i, d:], pos, rot["dims"], rot["base"])
        s = ((c @ uk[i].T) @ q[i, :d] + kr @ qr) * scale
        w = np.exp(s - s.max())
        w /= w.sum()
        out[i] = w @ (c @ uv[i].T)
    return W[p + "o"] @ out.reshape(-1)


def linear(W, name, h):
    return W[name] @ h + W[name + ".b"]


def chunk_attention(W, p, mx, state, cache, h, pos):
    """`cache`: state of the layer whose keys and values are read (its own, or an earlier layer's)."""
    H, G, d, dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = linear(W, p + "q", h).reshape(H, d)
    if cache is state:
        ks, vs = state.setdefault("k", []), state.setdefault("v", [])
        ks.append(np.stack([rotate_halves(r, pos, mx["rot"]) for r in linear(W, p + "k", h).reshape(G, d)]))
        vs.append(linear(W, p + "v", h).reshape(G, dv))
    first = pos // mx["mask"]["size"] * mx["mask"]["size"]
    k, v = np.stack(cache["k"][first:pos + 1]), np.stack(cache["v"][first:pos + 1])
    out = np.zeros((H, dv), dtype=h.dtype)
    for i in range(H):
        g = i // (H // G)
        s = k[:, g] @ rotate_halves(q[i], pos, mx["rot"]) * mx["scale"]
        w = np.exp(s - s.max())
        out[i] = (w / w.sum()) @ v[:, g]
    return linear(W, p + "o", out.reshape(-1) * sigmoid(W[p + "g"] @ h))


def mlstm_step(S, n, m, q, k, v, i, f):
    """One head, one token; i, f: logarithms of the gates.  Returns S [dim, vdim], n, m and the output."""
    new = max(f + m, i)
    keep, write = np.exp(f + m - new), np.exp(i - new)
    S = keep * S + write * np.outer(k, v)
    n = keep * n + write * k
    return S, n, new, S.T @ q / (max(abs(n @ q), np.exp(-new)) + 1e-6)


def mlstm_mixer(W, p, mx, eps, state, h):
    H, d, dv, cap = mx["heads"], mx["dim"], mx["vdim"], mx["gate_cap"]
    q = (W[p + "q"] @ h).reshape(H, d) * d ** -0.5
    k, v = (W[p + "k"] @ h).reshape(H, d), (W[p + "v"] @ h).reshape(H, dv)
    i = cap * np.tanh(linear(W, p + "i", h) / cap)
    f = -softplus(-cap * np.tanh(linear(W, p + "f", h) / cap))
    heads = state.setdefault("heads", [(np.zeros((d, dv), h.dtype), np.zeros(d, h.dtype), 0.0)] * H)
    new, out = [], np.zeros((H, dv), h.dtype)
    for x in range(H):
        S, n, m, out[x] = mlstm_step(*heads[x], q[x], k[x], v[x], i[x], f[x])
        new.append((S, n, m))
        out[x] = rms_norm(out[x], 1.0, eps)
    state["heads"] = new
    return W[p + "o"] @ (out.reshape(-1) * W[p + "norm"] * sigmoid(W[p + "g"] @ h))


# ---------------------------------------------------------------- feed-forward

def expert(W, p, h):
    return W[p + "down"] @ relu2(W[p + "up"] @ h)


def choose(scores, top):
    return np.argsort(-scores, kind="stable")[:top]


def moe(W, p, mlp, h):
    z = W[p + "router"] @ h
    s = np.exp(z - z.max())
    s /= s.sum()
    y = np.zeros_like(h)
    for e in choose(s, mlp["router"]["top"]):
        y = y + s[e] * expert(W, f"{p}e{e}.", h)
    if mlp.get("shared"):
        y = y + expert(W, p + "shared.", h)
    return y


# ---------------------------------------------------------------- the model

def new_state(cfg):
    return {"pos": 0, "layers": [{} for _ in cfg["layers"]]}


def copy_state(state):
    """Steps replace what a state holds and append to its lists; they never write into an array."""
    return {"pos": state["pos"], "layers": [{k: list(v) if isinstance(v, list) else v for k, v in L.items()} for L in state["layers"]]}


def step(cfg, W, state, token, trace=None):
    """One token through every layer; returns the logits.  `trace`: list that receives x after each layer."""
    return (step_norms_around if cfg["architecture"] == "Paposun" else step_one_norm)(cfg, W, state, token, trace)


def step_one_norm(cfg, W, state, token, trace):
    eps, pos = cfg["norm"]["eps"], state["pos"]
    x = W["embed"][token] * cfg["embedding"]["scale"]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = layer_norm(x, W[p + "norm1"], eps)
        st, mx = state["layers"][i], L["mixer"]
        if L["type"] == "latent_attention":
            y = latent_attention(W, p + "mix.", mx, eps, st, h, pos)
        else:
            y = delta_mixer(W, p + "mix.", mx, eps, L["type"] == "channel_delta", st, h, pos)
        if L.get("mlp"):
            y = y + moe(W, p + "mlp.", L["mlp"], h)
        x = x + y
        if trace is not None:
            trace.append(x.copy())
    state["pos"] = pos + 1
    return W["head"] @ layer_norm(x, W["final.norm"], eps)


def step_norms_around(cfg, W, state, token, trace):
    eps, pos, r = cfg["norm"]["eps"], state["pos"], cfg["residual_mult"]
    x = W["embed"][token]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = rms_norm(x, W[p + "norm1"], eps)
        st, mx = state["layers"][i], L["mixer"]
        if L["type"] == "attention":
            y = chunk_attention(W, p + "mix.", mx, st, state["layers"][mx["kv_from"]] if mx.get("kv_from") is not None else st, h, pos)
        else:
            y = mlstm_mixer(W, p + "mix.", mx, eps, st, h)
        x = x + r * rms_norm(y, W[p + "norm1b"], eps)
        if L.get("mlp"):
            y = W[p + "mlp.down"] @ gelu_tanh(W[p + "mlp.up"] @ rms_norm(x, W[p + "norm2"], eps))
            x = x + r * rms_norm(y, W[p + "norm2b"], eps)
        if trace is not None:
            trace.append(x.copy())
    state["pos"] = pos + 1
    return W["embed"] @ rms_norm(x, W["final.norm"], eps) * cfg["logit_scale"]


def run(cfg, W, tokens, state=None):
    """Logits at every token, [len(tokens), vocab]."""
    state = new_state(cfg) if state is None else state
    return np.stack([step(cfg, W, state, int(t)) for t in tokens])


def generate(cfg, W, prompt, n):
    """Greedy: the first maximum of the logits, n tokens."""
    state = new_state(cfg)
    for t in prompt:
        logits = step(cfg, W, state, int(t))
    out = [int(np.argmax(logits))]
    while len(out) < n:
        out.append(int(np.argmax(step(cfg, W, state, out[-1]))))
    return out
