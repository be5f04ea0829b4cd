"""A plain, slow restatement of the Suselorn decoder in numpy, one function per mechanism, for the
tests to compare the library with.  It shares no code with the product: tensors come in as a dict of
arrays, the configuration as the parsed config.json, and a whole sequence is recomputed every time
(no cache, no pages, no batch).  `dt` is the type everything is computed in."""
import numpy as np


def rms_norm(x, weight, eps):
    """x / sqrt(mean(x^2) + eps), times a plain weight."""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + x.dtype.type(eps)) * weight


def dyt_norm(x, alpha, weight, bias):
    """Dynamic Tanh: element by element, no statistics."""
    return np.tanh(alpha * x) * weight + bias


def rotate_pairs(x, pos, base, dims):
    """Interleaved rotation of the first `dims` entries of the last axis; pos broadcasts over x[..., 0].
    Pair i = entries (2i, 2i+1), angle pos * base^(-2i/dims) (angles in at least 32 bits)."""
    out = x.copy()
    for i in range(dims // 2):
        a = pos.astype(np.float64) * float(base) ** (-2.0 * i / dims)
        c, s = np.cos(a).astype(x.dtype), np.sin(a).astype(x.dtype)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def sink_softmax(scores, sink):
    """Softmax over the last axis whose denominator also holds exp(sink); -inf scores weigh nothing."""
    m = np.maximum(scores.max(-1, keepdims=True), sink)
    e = np.exp(scores - m)
    return e / (e.sum(-1, keepdims=True) + np.exp(sink - m))


def latent_attention(h, pos, w, cfg, eps):
    """h [T, width] -> [T, width].  w: this mixer's tensors by their last name part; keys and values are
    expanded from the latent, as the design states it (no absorbed products)."""
    H, dim, rot, vdim, rank = cfg["heads"], cfg["dim"], cfg["rot_dim"], cfg["vdim"], cfg["kv_rank"]
    T = h.shape[0]
    q = (rms_norm(h @ w["dq"].T, w["dq.norm"], eps) @ w["uq"].T).reshape(T, H, dim + rot)
    kv = h @ w["dkv"].T
    c = rms_norm(kv[:, :rank], w["dkv.norm"], eps)
    k_rot = rotate_pairs(kv[:, rank:], pos, cfg["rot"]["base"], cfg["rot"]["dims"])
    q_rot = rotate_pairs(q[:, :, dim:], pos[:, None], cfg["rot"]["base"], cfg["rot"]["dims"])
    k = (c @ w["uk"].T).reshape(T, H, dim)
    v = (c @ w["uv"].T).reshape(T, H, vdim)
    out = np.zeros((T, H, vdim), h.dtype)
    for head in range(H):
        s = (q[:, head, :dim] @ k[:, head].T + q_rot[:, head] @ k_rot.T) * h.dtype.type(cfg["scale"])
        s = np.where(pos[None, :] <= pos[:, None], s, -np.inf)
        out[:, head] = sink_softmax(s, w["sink"][head]) @ v[:, head]
    return out.reshape(T, H * vdim) @ w["o"].T


def gated_mlp(h, w):
    """silu gate, biases on all three projections."""
    g = h @ w["gate"].T + w["gate.b"]
    u = h @ w["up"].T + w["up.b"]
    return (g / (1 + np.exp(-g)) * u) @ w["down"].T + w["down.b"]


def hyper_read(streams, w_in):
    """streams [S, T, width] -> the sublayer's input [T, width]."""
    return np.einsum("s,std->td", w_in, streams)


def hyper_write(streams, mix, w_out, y):
    """mix[from, to]; every new stream from the old ones plus its share of the sublayer's result."""
    return np.einsum("st,sxd->txd", mix, streams) + w_out[:, None, None] * y[None]


def softcap(z, cap):
    return cap * np.tanh(z / cap)


def layer_runs(cfg):
    """Layer numbers in the order they run: the loop's span repeats, the rest follows."""
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return list(range(n))
    return list(range(loop["start"])) + list(range(loop["start"], loop["stop"])) * loop["times"] + list(range(loop["stop"], n))


def part(w, prefix):
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens, dt=np.float64, layers_out=None):
    """Logits [T, vocab] of one whole sequence; layers_out collects the sum of the streams after every layer run."""
    w = {k: np.asarray(v, dtype=dt) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    pos = np.arange(len(tokens))
    x = np.stack([w["embed"][np.asarray(tokens)]] * cfg["streams"])
    for i in layer_runs(cfg):
        L, p = cfg["layers"][i], f"l{i}."
        subs = [(1, lambda h: latent_attention(h, pos, part(w, p + "mix."), L["mixer"], eps))]
        if L.get("mlp"):
            subs.append((2, lambda h: gated_mlp(h, part(w, p + "mlp."))))
        for q, fn in subs:
            u = hyper_read(x, w[f"{p}hc{q}.in"])
            y = fn(dyt_norm(u, w[f"{p}norm{q}.alpha"], w[f"{p}norm{q}"], w[f"{p}norm{q}.b"])) * w[f"{p}ls{q}"]
            x = hyper_write(x, w[f"{p}hc{q}.mix"], w[f"{p}hc{q}.out"], y)
        if layers_out is not None:
            layers_out.append(x.sum(0))
    z = dyt_norm(x.sum(0), w["final.norm.alpha"], w["final.norm"], w["final.norm.b"])
    return softcap(z @ w["embed"].T, dt(cfg["logit_softcap"]))
