"""Plain, slow restatement of the Simivik design in numpy (float64): one function per mechanism, sharing no code with
the product.  A sequence at a time; x, h: [tokens, width]."""
import numpy as np


def rms(x, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def norm_around_zero(x, w, eps):
    """RMS norm whose stored weight is the distance from one."""
    return rms(x, eps) * (1.0 + w)


def causal_conv(u, taps):
    """u [tokens, channels], taps [channels, n]: the last tap meets the current token."""
    n = taps.shape[1]
    padded = np.concatenate([np.zeros((n - 1, u.shape[1])), u])
    out = np.zeros_like(u, dtype=np.float64)
    for j in range(n):
        out += taps[:, j] * padded[j:j + len(u)]
    return out


def rotate_half(x, positions, base, dims):
    """x [tokens, heads, dim]: dimension i turns with dimension i + dims/2; dimensions from `dims` on stay."""
    half = dims // 2
    angle = np.asarray(positions, np.float64)[:, None] * np.float64(base) ** (-2.0 * np.arange(half) / dims)
    c, s = np.cos(angle)[:, None, :], np.sin(angle)[:, None, :]
    out = np.array(x, np.float64)
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half] = u * c - v * s
    out[..., half:dims] = v * c + u * s
    return out


def visible(n, size, keep_first):
    """[query, key]: the last `size` keys, and the sequence's first ones."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep_first))


def window_attention(q, k, v, scale, cap, size, keep_first):
    """q [tokens, heads, dim], k [tokens, groups, dim], v [tokens, groups, vdim] -> [tokens, heads * vdim]."""
    n, heads = q.shape[:2]
    per = heads // k.shape[1]
    seen = visible(n, size, keep_first)
    out = np.zeros((n, heads, v.shape[2]))
    for h in range(heads):
        s = q[:, h] @ k[:, h // per].T * scale
        if cap is not None:
            s = cap * np.tanh(s / cap)
        s = np.where(seen, s, -np.inf)
        w = np.exp(s - s.max(1, keepdims=True))
        out[:, h] = w / w.sum(1, keepdims=True) @ v[:, h // per]
    return out.reshape(n, -1)


def decayed_state(q, k, v, decay, state=None):
    """q, k [tokens, heads, dim], v [tokens, heads, vdim] -> [tokens, heads, vdim] and the state [heads, dim, vdim]."""
    n, heads, dim = q.shape
    state = np.zeros((heads, dim, v.shape[2])) if state is None else np.array(state, np.float64)
    out = np.zeros(v.shape)
    for t in range(n):
        for h in range(heads):
            state[h] = decay[h] * state[h] + np.outer(k[t, h], v[t, h])
            out[t, h] = state[h].T @ q[t, h]
    return out, state


def route(z, top):
    """Router logits [tokens, experts] -> chosen experts [tokens, top] and their weights."""
    s = sigmoid(z)
    chosen = np.argsort(-s, axis=1, kind="stable")[:, :top]
    return chosen, np.take_along_axis(s, chosen, 1)


def gated(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def lightning_mixer(h, W, name, c, eps):
    H, n = c["heads"], len(h)
    q, k, v = (silu(h @ W[name + x].T).reshape(n, H, -1) for x in "qkv")
    o, _ = decayed_state(q, k, v, np.asarray(c["decay"], np.float64))
    o = rms(o.reshape(n, -1), eps) * W[name + "norm"]
    return (o * sigmoid(h @ W[name + "g"].T)) @ W[name + "o"].T


def attention_mixer(h, W, name, c):
    n = len(h)
    u = {x: h @ W[name + x].T for x in "qkv"}
    for x in u if c["conv"] else ():
        u[x] = causal_conv(u[x], W[name + x + ".conv"])
    q, k, v = u["q"].reshape(n, c["heads"], -1), u["k"].reshape(n, c["kv_heads"], -1), u["v"].reshape(n, c["kv_heads"], -1)
    q, k = (rotate_half(x, np.arange(n), c["rot"]["base"], c["rot"]["dims"]) for x in (q, k))
    return window_attention(q, k, v, c["scale"], c["softcap"], c["mask"]["size"], c["mask"]["keep_first"]) @ W[name + "o"].T


def dense_ff(h, W, name):
    return np.maximum(h @ W[name + "up"].T, 0.0) ** 2 @ W[name + "down"].T


def expert_ff(h, W, name, c):
    chosen, weight = route(h @ W[name + "router"].T, c["router"]["top"])
    out = np.zeros_like(h)
    for t in range(len(h)):
        for e, w in zip(chosen[t], weight[t]):
            out[t] += gated(w * h[t], *(W[f"{name}e{e}.{x}"] for x in ("gate", "up", "down")))
    if c.get("shared"):
        s = name + "shared."
        out += sigmoid(h @ W[s + "sg"].T) * gated(h, W[s + "gate"], W[s + "up"], W[s + "down"])
    return out


def source(layers, i):
    """The layer whose tensors layer i uses."""
    while layers[i].get("weights_of") is not None:
        i = layers[i]["weights_of"]
    return i


def forward(cfg, W, tokens, keep=None):
    """Logits [tokens, vocab]; `keep` collects the residual stream after every layer."""
    W = {n: np.asarray(a, np.float64) for n, a in W.items()}
    eps, layers = cfg["norm"]["eps"], cfg["layers"]
    x = W["embed"][np.asarray(tokens)]
    for i, layer in enumerate(layers):
        L = f"l{source(layers, i)}."
        h = norm_around_zero(x, W[L + "norm1"], eps)
        x = x + (lightning_mixer(h, W, L + "mix.", layer["mixer"], eps) if layer["type"] == "lightning"
                 else attention_mixer(h, W, L + "mix.", layer["mixer"]))
        mlp = layer.get("mlp")
        if mlp:
            h = norm_around_zero(x, W[L + "norm2"], eps)
            x = x + (dense_ff(h, W, L + "mlp.") if mlp["kind"] == "dense" else expert_ff(h, W, L + "mlp.", mlp))
        if keep is not None:
            keep.append(x)
    return norm_around_zero(x, W["final.norm"], eps) @ W["embed"].T
