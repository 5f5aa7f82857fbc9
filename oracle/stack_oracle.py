"""Plain restatement, in numpy and one token at a time, of a decoder whose layers are listed one by one (Nevurax):
short causal convolutions, the gated delta rule with one decay per head or per key channel, latent attention with a
sliding window and interleaved rotation, squared-ReLU experts behind a softmax router, one layer norm per layer whose
output both sublayers read.  Test infrastructure only: nothing here is used by the package, and nothing of the package
is used here.  Everything runs in the dtype of the weights handed in (float64 for pinning).

A model is a config dictionary (vocab, width, embedding.scale, norm.eps, layers[]: type, mixer, mlp) and a dictionary of
numpy arrays by tensor name.
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
