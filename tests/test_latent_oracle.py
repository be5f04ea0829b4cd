"""The plain restatement the GPU tests of the Suselorn design compare with: its own invariants, and that a mistake in
any one mechanism moves the logits of the test models by far more than the GPU tests tolerate.  CPU only."""
import ctypes as C
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from nvllm_amd import capi, synth
from tests import latent_oracle as O
from tests import latent_util as U


@pytest.mark.parametrize("name", sorted(U.CONFIGS))
def test_a_prefix_does_not_see_what_follows(tmp_path, name):
    _, cfg, w = U.model(tmp_path, name)
    seq = U.tokens(40, cfg["vocab"], 5)
    whole = O.forward(cfg, w, seq)
    assert U.error(O.forward(cfg, w, seq[:23]), whole[:23]) < 1e-12
    assert U.error(O.forward(cfg, w, seq, np.float32), whole) < 1e-5


def test_layer_order():
    cfg = dict(layers=[0] * 5, loop=dict(start=1, stop=3, times=3))
    assert O.layer_runs(cfg) == [0, 1, 2, 1, 2, 1, 2, 3, 4]
    assert O.layer_runs(dict(layers=[0] * 3, loop=None)) == [0, 1, 2]


def _planted(monkeypatch, name, value):
    monkeypatch.setattr(O, name, value)


def _rotate_halves(x, p, b, d, f=O.rotate_pairs):
    """Pairs (i, i + d/2) instead of neighbours."""
    order = np.stack([np.arange(d // 2), np.arange(d // 2) + d // 2], -1).ravel()
    out = np.empty_like(x)
    out[..., order] = f(x[..., order], p, b, d)
    return out


MISTAKES = {
    "no sink": lambda mp: _planted(mp, "sink_softmax", lambda s, k: np.exp(s - s.max(-1, keepdims=True)) / np.exp(s - s.max(-1, keepdims=True)).sum(-1, keepdims=True)),
    "rotation pairs halves": lambda mp: _planted(mp, "rotate_pairs", _rotate_halves),
    "position off by one per 16": lambda mp: _planted(mp, "rotate_pairs", lambda x, p, b, d, f=O.rotate_pairs: f(x, p + p // 16, b, d)),
    "eps outside the root": lambda mp: _planted(mp, "rms_norm", lambda x, w, e: x / (np.sqrt((x * x).mean(-1, keepdims=True)) + 0.05) * w),
    "mix transposed": lambda mp: _planted(mp, "hyper_write", lambda s, m, o, y, f=O.hyper_write: f(s, m.T, o, y)),
    "equal stream inputs": lambda mp: _planted(mp, "hyper_read", lambda s, i: s.mean(0)),
    "no norm bias": lambda mp: _planted(mp, "dyt_norm", lambda x, a, w, b, f=O.dyt_norm: f(x, a, w, 0 * b)),
    "no softcap": lambda mp: _planted(mp, "softcap", lambda z, c: z),
    "one run less": lambda mp: _planted(mp, "layer_runs", lambda c, f=O.layer_runs: f(c)[:-1]),
}


@pytest.mark.parametrize("mistake", sorted(MISTAKES))
def test_a_planted_mistake_shows(tmp_path, monkeypatch, mistake):
    _, cfg, w = U.model(tmp_path, "odd")
    seq = U.tokens(60, cfg["vocab"], 6)
    right = O.forward(cfg, w, seq)
    MISTAKES[mistake](monkeypatch)
    assert U.error(O.forward(cfg, w, seq), right) > 3 * U.limit(False), mistake


def test_absorbed_products_are_the_same_attention():
    """What the library computes (queries times W_uk against cached latents, attended latents times W_uv) is the design's
    attention: equal in exact arithmetic."""
    rng = np.random.Generator(np.random.PCG64(1))
    H, dim, vdim, rank, T = 3, 5, 7, 11, 9
    q, c = rng.standard_normal((T, H, dim)), rng.standard_normal((T, rank))
    uk, uv = rng.standard_normal((H, dim, rank)), rng.standard_normal((H, vdim, rank))
    p = np.tril(rng.random((T, T)))
    for h in range(H):
        np.testing.assert_allclose(q[:, h] @ (c @ uk[h].T).T, (q[:, h] @ uk[h]) @ c.T, rtol=1e-10, atol=1e-10)
        np.testing.assert_allclose(p @ (c @ uv[h].T), (p @ c) @ uv[h].T, rtol=1e-10, atol=1e-10)


def test_bf16_round_trip():
    a = np.array([1.0, -2.5, 3.1415927, 1e-30, 65280.0, 1.00390625], np.float32)
    b = synth.from_bf16(synth.to_bf16(a))
    assert np.all(np.abs(b - a) <= np.abs(a) * 2.0 ** -8)
    np.testing.assert_array_equal(synth.from_bf16(synth.to_bf16(b)), b)


def test_registry_and_replay_help():
    lib = capi.load_hip()
    assert lib.nvllm_has_architecture(b"Suselorn") == 1
    assert lib.nvllm_has_architecture(b"nothing of that name") == 0
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--help"], capture_output=True, text=True, timeout=60)
    assert r.returncode == 0 and "--max-tokens" in r.stdout
