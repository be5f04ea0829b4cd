"""Whole models of the Suselorn design through the library's own engine, block pool and scheduler, in bf16 and in fp32,
against the plain restatement on the same weights."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from nvllm_amd import capi, synth
from tests import latent_oracle as O
from tests import latent_util as U

pytestmark = pytest.mark.gpu
BOTH = pytest.mark.parametrize("f32", [True, False], ids=["fp32", "bf16"])


@BOTH
@pytest.mark.parametrize("name", sorted(U.CONFIGS))
def test_prompt_decode_and_portions(hip, tmp_path, name, f32):
    """The same tokens as one prompt, one by one, and in portions of many sizes down to two: the oracle's logits each time."""
    path, cfg, w = U.model(tmp_path, name)
    seq = U.tokens(150, cfg["vocab"], 11)
    want = O.forward(cfg, w, seq)
    eng = U.engine(hip, path, f32, tokens=160)
    plans = {
        "prompt": [[(0, 150)]],
        "tokens": [[(0, 1)] for _ in range(150)],
        "pairs": [[(0, 2)] for _ in range(75)],
        "portions": [[(0, n)] for n in (3, 16, 1, 17, 31, 2, 1, 33, 15, 2, 29)],
        "prompt, then decoding": [[(0, 70)]] + [[(0, 1)] for _ in range(80)],
    }
    worst = {}
    for what, plan in plans.items():
        assert sum(n for step in plan for _, n in step) == 150
        worst[what] = U.error(U.feed_all(eng, plan, {0: seq})[0], want)
    eng.close()
    assert max(worst.values()) < U.limit(f32), worst


@BOTH
def test_batches_of_unequal_requests(hip, tmp_path, f32):
    """Requests of unequal length and portions of prompts beside single tokens, in one batch, in slots and blocks that other
    requests have used before (the pool holds four requests at most): each as if it were alone."""
    path, cfg, w = U.model(tmp_path, "odd", seed=8)
    lengths = [1, 90, 2, 33, 64, 17, 100, 5, 48, 31]
    seqs = {i: U.tokens(n, cfg["vocab"], 100 + i) for i, n in enumerate(lengths)}
    r = np.random.Generator(np.random.PCG64(4))
    left, live, waiting, plan = dict(enumerate(lengths)), [], list(range(len(lengths))), []
    while waiting or live:
        while waiting and len(live) < 4:
            live.append(waiting.pop(0))
        step = []
        for q in live:
            if len(live) > 1 and r.random() < 0.2:
                continue                                  # left out of this step, goes on later
            n = min(left[q], int(r.choice([1, 1, 1, 2, 7, 16, 40])))
            step.append((q, n))
            left[q] -= n
        live = [q for q in live if left[q]]
        if step:
            plan.append(step)
    eng = U.engine(hip, path, f32, tokens=288)
    got = U.feed_all(eng, plan, seqs)
    assert capi.KVCacheManager.in_dll(hip.dll, "g_kv_manager").free_blocks_count == 18, "blocks were not given back"
    alone = {}
    for q, seq in seqs.items():
        alone[q] = U.feed_all(eng, [[(q, len(seq))]], {q: seq})[q]
    eng.close()
    for q, seq in seqs.items():
        want = O.forward(cfg, w, seq)
        assert U.error(got[q], want) < U.limit(f32), q
        assert U.error(alone[q], want) < U.limit(f32), q
        # (the two differ by the rounding of differently ordered sums only)
        assert U.error(got[q], alone[q]) < U.limit(f32), q


@BOTH
def test_a_far_key_across_blocks_and_slots(hip, tmp_path, f32):
    """One head's scores are raised until single keys decide: a long context, its last tokens decoded one by one."""
    def sharpen(name, v):
        return v * 2.5 if name.endswith(".uq") else (v - 8.0 if name.endswith(".sink") else None)
    cfg = synth.latent_config(64, 97, [(U.M(3, 32, 32, 32, 64, 48, base=50000.0), 64), (U.M(3, 32, 32, 32, 64, 48), 64)], loop=(0, 1, 2))
    path, cfg, w = U.model(tmp_path, "far", edit=sharpen, cfg=cfg)
    seq = U.tokens(700, 97, 2)
    want = O.forward(cfg, w, seq)
    weights = O.forward(cfg, w, np.concatenate([seq[:1], seq[2:]]))     # one early token less moves late logits: far keys matter
    assert U.error(weights[-200:], want[-200:]) > 3 * U.limit(False)
    eng = U.engine(hip, path, f32, tokens=704)
    whole = U.feed_all(eng, [[(0, 700)]], {0: seq})[0]
    cut = U.feed_all(eng, [[(0, 257)], [(0, 255)], [(0, 100)]] + [[(0, 1)] for _ in range(88)], {0: seq})[0]
    eng.close()
    lim = U.limit(f32) * (4 if f32 else 2)
    assert U.error(whole, want) < lim and U.error(cut, want) < lim, (U.error(whole, want), U.error(cut, want))


def test_prompt_of_the_dense_tile_size_in_bf16(hip, tmp_path):
    """256 tokens and more in one pass take the dense-tile projections, also block-diagonal ones; 600 tokens of two
    requests beside a decoded one."""
    for name in ("wide", "mixed", "heads33"):
        path, cfg, w = U.model(tmp_path, name, seed=5)
        seqs = {0: U.tokens(300, cfg["vocab"], 1), 1: U.tokens(299, cfg["vocab"], 2), 2: U.tokens(20, cfg["vocab"], 3)}
        eng = U.engine(hip, path, False, tokens=704)
        got = U.feed_all(eng, [[(2, 19)], [(0, 300), (2, 1), (1, 299)]], seqs)
        eng.close()
        for q, seq in seqs.items():
            assert U.error(got[q], O.forward(cfg, w, seq)) < U.limit(False), (name, q)


def test_long_decoding(hip, tmp_path):
    path, cfg, w = U.model(tmp_path, "mixed", seed=6)
    seq = U.tokens(400, cfg["vocab"], 9)
    want = O.forward(cfg, w, seq)
    eng = U.engine(hip, path, False, tokens=400)
    got = U.feed_all(eng, [[(0, 4)]] + [[(0, 1)] for _ in range(396)], {0: seq})[0]
    eng.close()
    assert U.error(got, want) < U.limit(False)


@BOTH
def test_unwanted_rows_and_bad_portions(hip, tmp_path, f32):
    path, cfg, w = U.model(tmp_path, "odd", seed=2)
    seq = U.tokens(60, cfg["vocab"], 1)
    want = O.forward(cfg, w, seq)
    eng = U.engine(hip, path, f32, slots=2, tokens=64)
    eng.feed(0, seq[:33])
    assert eng.feed_run().shape == (0, cfg["vocab"])     # nobody asked
    eng.feed(0, seq[33:50], [0, 5, 16])
    got = eng.feed_run()
    assert U.error(got, want[[33, 38, 49]]) < U.limit(f32)
    with pytest.raises(ValueError):
        eng.feed(0, [cfg["vocab"]])                      # no such token
    with pytest.raises(ValueError):
        eng.feed(0, seq[:15])                            # 65 positions
    with pytest.raises(ValueError, match="blocks"):
        eng.feed(1, seq[:16])                            # 50 positions hold all four blocks
    with pytest.raises(ValueError):
        eng.feed_run()                                   # nothing of the refused portions stayed
    eng.feed(0, seq[50:], [9])
    assert U.error(eng.feed_run(), want[59:]) < U.limit(f32)
    eng.feed_end(0)
    eng.feed(1, seq[:60], [59])
    assert U.error(eng.feed_run(), want[59:]) < U.limit(f32)
    eng.close()


def greedy(cfg, w, prompt, n):
    """Greedy continuation and, per generated token, how far the runner-up was (as a share of the logits' size)."""
    seq, margins = list(prompt), []
    for _ in range(n):
        z = O.forward(cfg, w, seq)[-1]
        top = np.sort(z)[-2:]
        margins.append((top[1] - top[0]) / np.sqrt((z * z).mean()))
        seq.append(int(z.argmax()))
    return seq, margins


@BOTH
@pytest.mark.parametrize("chunk,stepwise", [(0, False), (7, False), (16, True)])
def test_greedy_generation_through_the_scheduler(hip, tmp_path, monkeypatch, f32, chunk, stepwise):
    """set_request / step: arrival, chunked prefill, one token per sequence and step, with the next pass enqueued before
    the previous one is collected, and without; tokens as the oracle's as long as its choice is not a near tie."""
    if stepwise:
        monkeypatch.setenv("NVLLM_ENGINE_STEPWISE", "1")
    path, cfg, w = U.model(tmp_path, "odd", seed=12)
    prompts = [U.tokens(n, cfg["vocab"], 50 + n) for n in (1, 19, 40)]
    n_new = 14
    hip.nvllm_set_compute_dtype(capi.COMPUTE_F32 if f32 else capi.COMPUTE_BF16)
    for mode in (1, 0):
        hip.nvllm_set_logits_mode(mode)
        eng = capi.Engine(hip, path, 3, chunk_size=chunk, temperature=0.0, max_seq_len=64, recycle_blocks=1)
        for i, p in enumerate(prompts):
            eng.set_request(i, p, n_new, arrival_step=3 * i)
        eng.run_all()
        for i, p in enumerate(prompts):
            got = eng.history(i)
            want, margins = greedy(cfg, w, p, n_new)
            for k in range(n_new):
                if got[len(p) + k] != want[len(p) + k]:
                    assert margins[k] < (1e-4 if f32 else 0.2), (i, k, margins[k])
                    break                               # a near tie: the sequences part here
            else:
                k = n_new
            assert k >= 2 or margins[0] < 0.2, "the first tokens already differ"
        eng.close()
    hip.nvllm_set_logits_mode(0)


def test_sampling_with_a_temperature(hip, tmp_path):
    """sample() on this design's logits: a small temperature follows the maximum, and the same seed repeats itself."""
    path, cfg, w = U.model(tmp_path, "odd", seed=12)
    prompt = U.tokens(20, cfg["vocab"], 1)
    hip.nvllm_set_compute_dtype(capi.COMPUTE_F32)
    hip.nvllm_set_logits_mode(1)
    runs = []
    for temp in (1e-3, 1.0, 1.0):
        eng = capi.Engine(hip, path, 1, temperature=temp, topp=0.9, seed=7, max_seq_len=64)
        eng.set_request(0, prompt, 10)
        eng.run_all()
        runs.append(eng.history(0).tolist())
        eng.close()
    hip.nvllm_set_logits_mode(0)
    want, margins = greedy(cfg, w, prompt, 10)
    if min(margins) > 0.02:
        assert runs[0] == want
    assert runs[1] == runs[2]


def replay(tmp_path, path, steps, dtype, max_tokens):
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out = tmp_path / ("out_" + dtype)
    out.mkdir()
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", path, "--dtype", dtype, "--out", str(out), "--max-tokens", str(max_tokens)],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert r.stdout.split("\n")[:-1] == [f"done {s['step']}" for s in steps]
    return out


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_replaying_a_trace(tmp_path, dtype):
    path, cfg, w = U.model(tmp_path, "odd", seed=4)
    a, b = U.tokens(30, cfg["vocab"], 1).tolist(), U.tokens(9, cfg["vocab"], 2).tolist()
    steps = [dict(step=0, entries=[dict(id="a", tokens=a[:20], want=[19, 3])], end=[]),
             dict(step=1, entries=[dict(id="b", tokens=b, want=[]), dict(id="a", tokens=a[20:21], want=[])], end=["b"]),
             dict(step=2, entries=[dict(id="a", tokens=a[21:], want=[8]), dict(id="b", tokens=b, want=[8])], end=["a", "b"])]
    out = replay(tmp_path, path, steps, dtype, 64)
    za, zb = O.forward(cfg, w, a), O.forward(cfg, w, b)
    V, lim = cfg["vocab"], U.limit(dtype == "float32")
    assert U.error(np.fromfile(out / "0.f32", "<f4").reshape(-1, V), za[[19, 3]]) < lim
    assert not (out / "1.f32").exists()
    assert U.error(np.fromfile(out / "2.f32", "<f4").reshape(-1, V), np.stack([za[29], zb[8]])) < lim


def test_generating_from_the_command_line(tmp_path, tmp_models):
    """The same command generates from a folder and from a model file."""
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    path, cfg, w = U.model(tmp_path, "mixed", seed=4)

    def run(model, vocab, *more):
        prompts = [U.tokens(n, vocab, n).tolist() for n in (3, 11)]
        r = subprocess.run([os.path.join(root, "bin", "generate"), "--model", model, "-n", "6"] + [f"--prompt={','.join(map(str, p))}" for p in prompts] +
                           list(more), capture_output=True, text=True, timeout=100)
        assert r.returncode == 0, r.stderr[-2000:]
        lines = [[[int(t) for t in part.split(",")] for part in line.split("|")] for line in r.stdout.strip().split("\n")]
        assert [l[0] for l in lines] == prompts and all(len(l[1]) == 6 for l in lines)
        return lines
    for prompt, new in run(path, cfg["vocab"], "--dtype", "float32"):
        want, margins = greedy(cfg, w, prompt, 6)
        assert new == want[len(prompt):] or min(margins) < 1e-4
    file_path, shape = tmp_models("tiny")
    run(file_path, shape.vocab_size, "--chunk-size", "4")


def test_a_pool_of_another_model_is_refused(hip, tmp_path):
    """init_kv_cache_manager, all an older driver knows, makes the loaded folder model's pool; nothing else fits it."""
    import ctypes as C
    path, cfg, w = U.model(tmp_path, "mixed", seed=4)
    hip.nvllm_set_compute_dtype(capi.COMPUTE_BF16)
    weights, config = capi.Weights(), capi.Config()
    hip.load_model(C.byref(weights), C.byref(config), path.encode())
    sizes = []
    for make in (lambda m: hip.init_kv_cache_manager(C.byref(m), 16, 8, config.n_layers, config.n_kv_heads, config.head_dim),
                 lambda m: hip.nvllm_init_model_kv(C.byref(m), 16, 8, C.byref(config), C.byref(weights)),
                 lambda m: hip.init_kv_cache_manager(C.byref(m), 16, 8, 1, 2, 16)):
        mgr = capi.KVCacheManager()
        make(mgr)
        sizes.append((bool(mgr.pool_k), bool(mgr.pool_v), mgr.free_blocks_count))
        hip.free_kv_cache_manager(C.byref(mgr))
    assert sizes == [(True, False, 8), (True, False, 8), (True, True, 8)]
    hip.nvllm_free_model(C.byref(weights))


@pytest.mark.parametrize("what", ["mixer", "architecture", "shape", "loop"])
def test_a_folder_that_does_not_fit_is_refused(tmp_path, what):
    """Configurations the library does not know, or that the tensors contradict, end with a message and an error status."""
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    path, cfg, _ = U.model(tmp_path, "mixed", seed=4)
    cfg = json.loads(json.dumps(cfg))
    if what == "mixer":
        cfg["layers"][1]["type"] = "something_else"
    elif what == "architecture":
        cfg["architecture"] = "Unheardof"
    elif what == "shape":
        cfg["layers"][0]["mixer"]["kv_rank"] += 16
    else:
        cfg["loop"] = dict(start=1, stop=9, times=2)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    r = subprocess.run([os.path.join(root, "bin", "generate"), "--model", path, "-n", "1"], capture_output=True, text=True, timeout=100)
    assert r.returncode != 0 and r.stdout == ""
    assert {"mixer": "something_else", "architecture": "Unheardof", "shape": "asks for", "loop": "loop"}[what] in r.stderr
