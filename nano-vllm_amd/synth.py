"""Synthetic model files, tokenizer files and request sets in the reference's formats.

No real checkpoints exist offline, so every test and benchmark runs on random-init
files of the published shapes.  The formats are the reference's:

* ``model.bin``: 7 int32 header (dim, hidden_dim, n_layers, n_heads, n_kv_heads,
  vocab_size, max_seq_len) followed by the tensors grouped by kind across layers
  in the order the loader reads them -- embed, rms_att[L], wq[L], wk[L], wv[L],
  wo[L], rms_ffn[L], w_gate[L], w_down[L], w_up[L], rms_final, (lm_head)
  (reference src/model.c:118,230-279).
* ``tokenizer.bin``: int32 max_token_length, then per token float32 score, int32
  length, bytes (reference src/tokenizer.c:43-77).

Values are small integers over a power of two, hence exactly representable in
fp16: an fp16 file and the fp32 expansion the reference makes of it hold the same
numbers.  Generation is seeded and chunked so that a 1.1 B-parameter file needs
little memory.
"""
from __future__ import annotations

import os
import struct
from dataclasses import dataclass

import numpy as np

SHAPES = {
    # name: dim, hidden_dim, n_layers, n_heads, n_kv_heads, vocab_size, max_seq_len
    "tiny": (64, 160, 2, 4, 2, 512, 128),
    "tiny-mha48": (96, 224, 2, 2, 2, 384, 96),        # head_dim 48, like stories15M
    "tiny-gqa": (256, 512, 3, 8, 4, 600, 160),        # grouped heads that divide over 2 or 4 tensor-parallel ranks
    "stories15M": (288, 768, 6, 6, 6, 32000, 256),
    "stories42M": (512, 1376, 8, 8, 8, 32000, 1024),
    "tinyllama-1.1b": (2048, 5632, 22, 32, 4, 32000, 2048),
    "llama2-7b": (4096, 11008, 32, 32, 32, 32000, 2048),
}


@dataclass
class ModelShape:
    dim: int
    hidden_dim: int
    n_layers: int
    n_heads: int
    n_kv_heads: int
    vocab_size: int
    max_seq_len: int

    @property
    def head_dim(self) -> int:
        return self.dim // self.n_heads

    @classmethod
    def named(cls, name: str, **over) -> "ModelShape":
        s = cls(*SHAPES[name])
        for k, v in over.items():
            setattr(s, k, v)
        return s

    def header(self) -> bytes:
        return struct.pack("<7i", self.dim, self.hidden_dim, self.n_layers, self.n_heads,
                           self.n_kv_heads, self.vocab_size, self.max_seq_len)

    def n_params(self, shared: bool = False) -> int:
        D, F, L, V = self.dim, self.hidden_dim, self.n_layers, self.vocab_size
        QD, KD = self.n_heads * self.head_dim, self.n_kv_heads * self.head_dim
        body = V * D + L * (2 * D + D * QD + 2 * D * KD + QD * D + 3 * D * F) + D
        return body if shared else body + V * D


_CHUNK = 1 << 24


def _write_random(f, n: int, rng: np.random.Generator, span: int, denom: float, dtype, noise=None) -> None:
    """n values k/denom with k uniform in [-span, span], streamed in chunks.  With a
    `noise` generator every value also gets a relative perturbation of about 1e-4, which
    takes it off the fp16 grid (fp32 files only)."""
    done = 0
    while done < n:
        m = min(_CHUNK, n - done)
        k = rng.integers(-span, span + 1, size=m, dtype=np.int16)
        v = k.astype(np.float32) / np.float32(denom)
        if noise is not None:
            v = v + noise.standard_normal(m).astype(np.float32) * np.float32(span / denom * 1e-4)
        v.astype(dtype).tofile(f)
        done += m


def _write_norm(f, n: int, rng: np.random.Generator, dtype) -> None:
    """RMSNorm gains near one: 1 + k/64, k in [-8, 8]."""
    k = rng.integers(-8, 9, size=n, dtype=np.int16)
    (1.0 + k.astype(np.float32) / 64.0).astype(dtype).tofile(f)


def write_model(path: str, shape: ModelShape, seed: int = 0, dtype: str = "f16",
                shared: bool = False, rope_tail: bool = False, progress=None, exact16: bool = True) -> int:
    """Write a random-init model file; returns its size in bytes.

    Matrices: k/4096 with |k| <= 82 (about +-0.02); embedding (and a separate
    classifier): k/128 with |k| <= 64 (about +-0.5); norm gains 1 + k/64.
    ``rope_tail`` appends the legacy llama2.c RoPE tables (fp32 shared files only).
    ``progress(name)`` is called after every tensor kind (large files take a while).
    ``exact16=False`` (fp32 files) perturbs every matrix value so that fp16 cannot hold it,
    like the weights of a trained fp32 checkpoint.
    """
    progress = progress or (lambda name: None)
    np_dtype = {"f16": np.float16, "f32": np.float32}[dtype]
    D, F, L, V = shape.dim, shape.hidden_dim, shape.n_layers, shape.vocab_size
    QD, KD = shape.n_heads * shape.head_dim, shape.n_kv_heads * shape.head_dim
    rng = np.random.Generator(np.random.PCG64(seed))
    noise = None
    if not exact16:
        assert dtype == "f32", "only an fp32 file can hold values off the fp16 grid"
        noise = np.random.Generator(np.random.PCG64(seed + 104729))
    tmp = path + ".tmp"
    with open(tmp, "wb") as f:
        f.write(shape.header())
        _write_random(f, V * D, rng, 64, 128.0, np_dtype, noise)       # token_embedding_table
        for _ in range(L):
            _write_norm(f, D, rng, np_dtype)                           # rms_att_weight
        for name, n in (("wq", D * QD), ("wk", D * KD), ("wv", D * KD), ("wo", QD * D)):
            for _ in range(L):
                _write_random(f, n, rng, 82, 4096.0, np_dtype, noise)
            progress(name)
        for _ in range(L):
            _write_norm(f, D, rng, np_dtype)                           # rms_ffn_weight
        for name, n in (("w_gate", D * F), ("w_down", F * D), ("w_up", D * F)):
            for _ in range(L):
                _write_random(f, n, rng, 82, 4096.0, np_dtype, noise)
            progress(name)
        _write_norm(f, D, rng, np_dtype)                               # rms_final_weight
        if not shared:
            _write_random(f, V * D, rng, 64, 2048.0, np_dtype, noise)  # lm_head
        if rope_tail:
            assert dtype == "f32" and shared
            np.zeros(shape.max_seq_len * shape.head_dim, np.float32).tofile(f)
    os.replace(tmp, path)
    return os.path.getsize(path)


def write_tokenizer(path: str, vocab_size: int) -> None:
    """A tokenizer file the reference's BPE encoder can digest: ids 0-2 specials,
    3-258 the byte tokens '<0xNN>', then ' ' and printable single characters, then
    unique filler strings (so decoded text is invertible to ids)."""
    pieces = ["<unk>", "<s>", "</s>"] + [f"<0x{b:02X}>" for b in range(256)]
    singles = [" "] + [chr(c) for c in range(33, 127)]
    pieces += singles
    i = 0
    while len(pieces) < vocab_size:
        pieces.append(f"▁t{i}")
        i += 1
    pieces = pieces[:vocab_size]
    enc = [p.encode("utf-8") for p in pieces]
    with open(path, "wb") as f:
        f.write(struct.pack("<i", max(len(e) for e in enc)))
        for e in enc:
            f.write(struct.pack("<fi", 0.0, len(e)))
            f.write(e)


def make_requests(n: int, prompt_lo: int, prompt_hi: int, vocab_size: int, seed: int = 0,
                  bos: int = 1):
    """n prompts of token ids in [3, vocab) with BOS first (reference
    src/tokenizer.c:136), lengths uniform in [prompt_lo, prompt_hi]."""
    rng = np.random.Generator(np.random.PCG64(seed + 7919))
    out = []
    for _ in range(n):
        ln = int(rng.integers(prompt_lo, prompt_hi + 1))
        p = rng.integers(3, vocab_size, size=ln, dtype=np.int64).astype(np.int32)
        p[0] = bos
        out.append(p)
    return out


# ------------------------------------------------------------------ model folders
# config.json + model.safetensors (random bf16 weights) of the "Suselorn" and "Simivik" designs.  Test-sized models
# come with weights that make every mechanism matter (attention scores of several units, sinks of their size, streams
# that mix, routers without close calls); `plain=True` writes the same tensors from one repeated random block, for benchmark-sized files.

def latent_mixer(heads, dim, rot_dim, vdim, kv_rank, q_rank, scale=None, base=10000.0) -> dict:
    return dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank,
                scale=float(scale if scale is not None else (dim + rot_dim) ** -0.5), rot=dict(base=float(base), dims=rot_dim))


def latent_config(width, vocab, layers, streams=2, loop=None, softcap=20.0, eps=1e-5) -> dict:
    """layers: (mixer dict, ff width or None) per layer; loop: (start, stop, times) or None."""
    return dict(architecture="Suselorn", width=width, vocab=vocab, streams=streams, logit_softcap=softcap, norm=dict(eps=eps),
                loop=None if loop is None else dict(start=loop[0], stop=loop[1], times=loop[2]),
                layers=[dict(type="latent_attention", mixer=m, mlp=None if ff is None else dict(kind="dense", ff=ff)) for m, ff in layers])


def latent_tensors(cfg: dict) -> dict:
    """name -> (shape, kind) of every tensor of the design, in file order."""
    D, S = cfg["width"], cfg["streams"]
    out = {"embed": ((cfg["vocab"], D), "embed")}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        H, parts = m["heads"], (1, 2) if layer["mlp"] else (1,)
        for q in parts:
            out[f"{p}norm{q}"] = ((D,), "gain")
            out[f"{p}norm{q}.b"] = ((D,), "bias")
            out[f"{p}norm{q}.alpha"] = ((), "alpha")
        x = p + "mix."
        out[x + "dq"] = ((m["q_rank"], D), "matrix")
        out[x + "dq.norm"] = ((m["q_rank"],), "gain")
        out[x + "uq"] = ((H * (m["dim"] + m["rot_dim"]), m["q_rank"]), "sharp")
        out[x + "dkv"] = ((m["kv_rank"] + m["rot_dim"], D), "matrix")
        out[x + "dkv.norm"] = ((m["kv_rank"],), "gain")
        out[x + "uk"] = ((H * m["dim"], m["kv_rank"]), "sharp")
        out[x + "uv"] = ((H * m["vdim"], m["kv_rank"]), "matrix")
        out[x + "sink"] = ((H,), "sink")
        out[x + "o"] = ((D, H * m["vdim"]), "matrix")
        if layer["mlp"]:
            ff, x = layer["mlp"]["ff"], p + "mlp."
            for n, shape in (("gate", (ff, D)), ("up", (ff, D)), ("down", (D, ff))):
                out[x + n] = (shape, "matrix")
                out[x + n + ".b"] = ((shape[0],), "bias")
        for q in parts:
            out[f"{p}ls{q}"] = ((D,), "gain")
            out[f"{p}hc{q}.in"] = ((S,), "weight")
            out[f"{p}hc{q}.out"] = ((S,), "weight")
            out[f"{p}hc{q}.mix"] = ((S, S), "mix")
    out["final.norm"] = ((D,), "gain")
    out["final.norm.b"] = ((D,), "bias")
    out["final.norm.alpha"] = ((), "alpha")
    return out


def lightning_mixer(heads, dim, vdim, decay=None) -> dict:
    """decay: one number per head; default: half-lives from about a token to hundreds."""
    if decay is None:
        decay = [float(np.exp(-0.7 * 0.35 ** i)) for i in range(heads)]
    return dict(heads=heads, dim=dim, vdim=vdim, decay=[float(d) for d in decay])


def window_mixer(heads, kv_heads, dim, vdim, size, keep_first, taps=4, rot=None, base=10000.0, scale=None, softcap=25.0) -> dict:
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=taps, mask=dict(size=size, keep_first=keep_first), softcap=softcap,
                rot=dict(base=float(base), dims=dim if rot is None else rot), scale=float(dim ** -0.5 if scale is None else scale))


def expert_mlp(ff, experts, top, shared_ff=None) -> dict:
    return dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top), shared=None if shared_ff is None else dict(ff=shared_ff))


def hybrid_config(width, vocab, layers, eps=1e-5) -> dict:
    """layers: (mixer dict, feed-forward) per layer -- the feed-forward a width (dense), an expert_mlp() or None -- or the
    index of the layer whose tensors it shares."""
    out = []
    for layer in layers:
        if isinstance(layer, int):
            out.append(dict(out[layer], weights_of=layer))
            continue
        mixer, mlp = layer
        out.append(dict(type="lightning" if "decay" in mixer else "attention", mixer=mixer, mlp=dict(kind="dense", ff=mlp) if isinstance(mlp, int) else mlp))
    return dict(architecture="Simivik", width=width, vocab=vocab, norm=dict(eps=eps), layers=out)


def hybrid_tensors(cfg: dict) -> dict:
    D = cfg["width"]
    out = {"embed": ((cfg["vocab"], D), "routed_embed")}
    for i, layer in enumerate(cfg["layers"]):
        if "weights_of" in layer:
            continue
        p, m, mlp = f"l{i}.", layer["mixer"], layer["mlp"]
        out[p + "norm1"] = ((D,), "routed_zero_gain")
        if mlp:
            out[p + "norm2"] = ((D,), "routed_zero_gain")
        x, H = p + "mix.", m["heads"]
        G = m.get("kv_heads", H)
        sizes = dict(q=H * m["dim"], k=G * m["dim"], v=G * m["vdim"])
        for n, rows in sizes.items():
            out[x + n] = ((rows, D), "matrix" if n == "v" else "sharp")
        if layer["type"] == "lightning":
            out[x + "g"] = ((H * m["vdim"], D), "matrix")
            out[x + "norm"] = ((H * m["vdim"],), "gain")
        elif m["conv"]:
            for n, rows in sizes.items():
                out[f"{x}{n}.conv"] = ((rows, m["conv"]), "taps")
        out[x + "o"] = ((D, H * m["vdim"]), "routed_out")
        x = p + "mlp."
        if mlp and mlp["kind"] == "dense":
            out[x + "up"], out[x + "down"] = ((mlp["ff"], D), "matrix"), ((D, mlp["ff"]), "routed_out")
        elif mlp:
            parts = [(f"{x}e{e}.", mlp["expert"]["ff"]) for e in range(mlp["router"]["experts"])]
            if mlp.get("shared"):
                parts.append((x + "shared.", mlp["shared"]["ff"]))
                out[x + "shared.sg"] = ((1, D), "matrix")
            for n, ff in parts:
                out[n + "gate"], out[n + "up"], out[n + "down"] = ((ff, D), "matrix"), ((ff, D), "matrix"), ((D, ff), "routed_out")
            out[x + "router"] = ((mlp["router"]["experts"], D), "router")
    out["final.norm"] = ((D,), "zero_gain")
    return out


def _routed_dims(cfg) -> int:
    """The first dims of the residual belong to the routers of test-sized models: a token's embedding holds its experts' order
    there, well apart, and no layer writes to them -- so that the choice never hangs on rounding."""
    return max([l["mlp"]["router"]["experts"] for l in cfg.get("layers", []) if l.get("mlp") and l["mlp"]["kind"] == "moe"], default=0)


DESIGN_TENSORS = {"Suselorn": latent_tensors, "Simivik": hybrid_tensors}


def to_bf16(a: np.ndarray) -> np.ndarray:
    """fp32 -> bf16 bit patterns, to nearest even."""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def from_bf16(u: np.ndarray) -> np.ndarray:
    return (u.astype(np.uint32) << 16).view(np.float32)


def _tensor_values(shape, kind, rng, routed=0) -> np.ndarray:
    if kind.startswith("routed_"):
        v = _tensor_values(shape, kind[7:], rng)
        if kind == "routed_embed" and routed:   # every row a permutation of evenly spaced numbers
            v[:, :routed] = (rng.permuted(np.tile(np.arange(routed), (shape[0], 1)), axis=1) - (routed - 1) / 2)
        else:
            v[:routed] = 0.0
        return v
    n = rng.standard_normal(shape)
    fan = shape[-1] if shape else 1
    return {"embed": lambda: n, "matrix": lambda: n * fan ** -0.5, "sharp": lambda: n * 1.7 * fan ** -0.5,
            "gain": lambda: 1.0 + 0.2 * n, "bias": lambda: 0.2 * n, "alpha": lambda: 0.6 + 0.2 * rng.random(shape),
            "sink": lambda: 1.5 + 2.0 * n, "weight": lambda: 0.4 + 0.8 * rng.random(shape),
            "mix": lambda: 0.9 * np.eye(fan) + 0.2 * n, "zero_gain": lambda: 0.2 * n, "out": lambda: n * fan ** -0.5,
            "taps": lambda: 0.4 * n + np.eye(fan)[-1], "router": lambda: np.eye(*shape) * 1.5 + 0.005 * n}[kind]()


def write_model_dir(path: str, cfg: dict, seed: int = 0, plain: bool = False, edit=None) -> dict:
    """Write config.json and model.safetensors into folder `path`; returns the tensors (as fp32, exactly what the file
    holds; none with `plain`).  `edit(name, array)` may return a replacement for a tensor's values before rounding."""
    import json
    os.makedirs(path, exist_ok=True)
    rng = np.random.Generator(np.random.PCG64(seed))
    tensors, routed = DESIGN_TENSORS[cfg["architecture"]](cfg), _routed_dims(cfg)
    header, at = {}, 0
    for name, (shape, _) in tensors.items():
        size = 2 * int(np.prod(shape, dtype=np.int64))
        header[name] = dict(dtype="BF16", shape=list(shape), data_offsets=[at, at + size])
        at += size
    text = json.dumps(header).encode()
    text += b" " * (-len(text) % 8)
    out = {}
    block = rng.standard_normal(1 << 22).astype(np.float32) if plain else None
    tmp = os.path.join(path, "model.safetensors.tmp")
    with open(tmp, "wb") as f:
        f.write(struct.pack("<Q", len(text)))
        f.write(text)
        for name, (shape, kind) in tensors.items():
            if plain and kind in ("embed", "routed_embed", "matrix", "sharp", "routed_out", "router"):
                scale = 1.0 if kind.endswith("embed") else shape[-1] ** -0.5
                chunk, left = to_bf16(block * np.float32(scale)), int(np.prod(shape, dtype=np.int64))
                while left > 0:
                    chunk[:min(left, len(chunk))].tofile(f)
                    left -= len(chunk)
                continue
            v = np.asarray(_tensor_values(shape, kind, rng, 0 if plain else routed), np.float32)
            if edit is not None:
                new = edit(name, v)
                v = v if new is None else np.asarray(new, np.float32)
            bits = to_bf16(v.reshape(shape))
            bits.tofile(f)
            if not plain:
                out[name] = from_bf16(bits)
    os.replace(tmp, os.path.join(path, "model.safetensors"))
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f, indent=1)
    return out
