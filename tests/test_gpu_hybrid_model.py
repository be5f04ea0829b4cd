"""Whole models of the Simivik design through the library's own engine, block pool, state slots and scheduler, in bf16 and
in fp32, against the plain restatement on the same weights."""
import json
import os
import subprocess

import numpy as np
import pytest

from nvllm_amd import capi, synth
from tests import hybrid_oracle as O
from tests import hybrid_util as U
from tests.test_gpu_latent_model import replay

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
@pytest.mark.parametrize("name", ["odd", "parts"])
def test_batches_of_unequal_requests(hip, tmp_path, name, f32):
    """Requests of unequal length and portions of prompts beside single tokens, in one batch, in slots and blocks that other
    requests have used before (the pool holds four requests at most): each as if it were alone."""
    path, cfg, w = U.model(tmp_path, name, seed=8)
    lengths = [1, 90, 2, 33, 64, 17, 100, 5, 48, 31, 3, 70]
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
    alone = {q: U.feed_all(eng, [[(q, len(seq))]], {q: seq})[q] for q, seq in seqs.items()}
    eng.close()
    for q, seq in seqs.items():
        want = O.forward(cfg, w, seq)
        assert U.error(got[q], want) < U.limit(f32), q
        assert U.error(alone[q], want) < U.limit(f32), q
        assert U.error(got[q], alone[q]) < U.limit(f32), q   # (the two differ by rounding only)


@BOTH
def test_far_keys_and_window_edges(hip, tmp_path, f32):
    """Sharpened scores: single keys decide -- kept first tokens hundreds of tokens back, the window's last key -- in prompts and in
    decoding; a decay near one carries early tokens far beside them."""
    def sharpen(name, v):
        return v * 2.0 if name.endswith(("mix.q", "mix.k")) and v.shape[0] != 128 else None
    cfg = synth.hybrid_config(64, 97, [(U.A(4, 2, 32, 32, size=70, keep_first=5, taps=2, base=50000.0, softcap=28.0), 64), (U.L(4, 32, 32, [0.999, 0.99, 0.9, 0.5]), 64),
                                       (U.A(4, 1, 32, 32, size=33, keep_first=18, taps=4, rot=16), 64)])
    path, cfg, w = U.model(tmp_path, "far", edit=sharpen, cfg=cfg)
    seq = U.tokens(700, 97, 2)
    want = O.forward(cfg, w, seq)
    other = O.forward(cfg, w, np.concatenate([(seq[:2] + 1) % 97, seq[2:]]))      # two early tokens move late logits: far tokens matter
    assert U.error(other[-200:], want[-200:]) > 3 * U.limit(False)
    eng = U.engine(hip, path, f32, tokens=704)
    whole = U.feed_all(eng, [[(0, 700)]], {0: seq})[0]
    cut = U.feed_all(eng, [[(0, 257)], [(0, 255)], [(0, 100)]] + [[(0, 1)] for _ in range(88)], {0: seq})[0]
    eng.close()
    lim = U.limit(f32) * (4 if f32 else 2)
    assert U.error(whole, want) < lim and U.error(cut, want) < lim, (U.error(whole, want), U.error(cut, want))


@pytest.mark.parametrize("name", ["odd", "parts", "edges", "groups"])
def test_prompts_of_the_dense_tile_size_in_bf16(hip, tmp_path, name):
    """256 tokens and more in one pass take the dense-tile projections, the experts' too; 600 tokens of two requests beside a
    decoded one."""
    path, cfg, w = U.model(tmp_path, name, seed=5)
    seqs = {0: U.tokens(300, cfg["vocab"], 1), 1: U.tokens(299, cfg["vocab"], 2), 2: U.tokens(20, cfg["vocab"], 3)}
    eng = U.engine(hip, path, False, tokens=704)
    got = U.feed_all(eng, [[(2, 19)], [(0, 300), (2, 1), (1, 299)]], seqs)
    eng.close()
    for q, seq in seqs.items():
        assert U.error(got[q], O.forward(cfg, w, seq)) < U.limit(False), (name, q)


@BOTH
def test_long_decoding(hip, tmp_path, f32):
    path, cfg, w = U.model(tmp_path, "parts", seed=6)
    seq = U.tokens(400, cfg["vocab"], 9)
    want = O.forward(cfg, w, seq)
    eng = U.engine(hip, path, f32, tokens=400)
    got = U.feed_all(eng, [[(0, 4)]] + [[(0, 1)] for _ in range(396)], {0: seq})[0]
    eng.close()
    assert U.error(got, want) < U.limit(f32)


def test_widths_that_are_not_padded_and_one_expert_for_all(hip, tmp_path):
    """Every width a multiple of what the tiles want, and all experts chosen: nothing rests on padding or on a free expert."""
    cfg = synth.hybrid_config(128, 256, [(U.L(4, 32, 64), U.E(64, 2, 2, 64)), (U.A(8, 4, 64, 64, size=24, keep_first=8), 256)])
    path, cfg, w = U.model(tmp_path, "round", cfg=cfg)
    seq = U.tokens(90, 256, 3)
    want = O.forward(cfg, w, seq)
    for f32 in (True, False):
        eng = U.engine(hip, path, f32, tokens=96)
        for plan in ([[(0, 90)]], [[(0, 50)], [(0, 2)]] + [[(0, 1)]] * 38):
            assert U.error(U.feed_all(eng, plan, {0: seq})[0], want) < U.limit(f32)
        eng.close()


@BOTH
def test_blocks_of_other_sizes(hip, tmp_path, f32):
    path, cfg, w = U.model(tmp_path, "odd", seed=2)
    seq = U.tokens(100, cfg["vocab"], 1)
    want = O.forward(cfg, w, seq)
    hip.nvllm_set_compute_dtype(capi.COMPUTE_F32 if f32 else capi.COMPUTE_BF16)
    hip.nvllm_set_logits_mode(0)
    for bs in (32, 48) + ((10,) if f32 else ()):
        eng = capi.Engine(hip, path, 2, block_size=bs, max_seq_len=110, max_steps=1 << 30)
        assert U.error(U.feed_all(eng, [[(0, 60)], [(0, 3)]] + [[(0, 1)]] * 37, {0: seq})[0], want) < U.limit(f32), bs
        eng.close()


@BOTH
def test_more_sequences_than_the_states_were_made_for(hip, tmp_path, f32):
    """The states' memory grows when a pass brings a sequence id it has no slot for; what the others carry stays."""
    import ctypes as C
    path, cfg, w = U.model(tmp_path, "odd", seed=4)
    seq = U.tokens(24, cfg["vocab"], 8)
    want = O.forward(cfg, w, seq)
    hip.nvllm_set_compute_dtype(capi.COMPUTE_F32 if f32 else capi.COMPUTE_BF16)
    hip.nvllm_set_logits_mode(0)
    mgr = capi.KVCacheManager.in_dll(hip.dll, "g_kv_manager")
    tables = [(C.c_int * 2)(0, 1), (C.c_int * 2)(2, 3)]
    empty = capi.BlockTable(C.cast(tables[0], capi.c_int_p), 0)
    both = [capi.BlockTable(C.cast(t, capi.c_int_p), 2) for t in tables]
    ptrs = (C.POINTER(capi.BlockTable) * 6)(*[C.pointer(both[0] if i == 0 else both[1] if i == 5 else empty) for i in range(6)])
    weights, config, state = capi.Weights(), capi.Config(), capi.RunState()
    hip.load_model(C.byref(weights), C.byref(config), path.encode())
    config.max_seq_len = 64
    hip.malloc_run_state(C.byref(state), C.byref(config))
    hip.nvllm_init_model_kv(C.byref(mgr), 16, 8, C.byref(config), C.byref(weights))
    got = {0: [], 5: []}

    def run(parts):
        toks, pos, ids = [], [], []
        for s, a, b in parts:
            toks += seq[a:b].tolist()
            pos += list(range(a, b))
            ids += [s] * (b - a)
        n = len(toks)
        hip.transformer_batch(capi.ints(toks), n, capi.ints(pos), capi.ints(ids), capi.ints(range(n)), n, C.byref(config), C.byref(state), C.byref(weights), ptrs)
        rows = np.ctypeslib.as_array(C.cast(state.logits, C.POINTER(C.c_float)), (n * cfg["vocab"],)).reshape(n, -1).copy()
        at = 0
        for s, a, b in parts:
            got[s].append(rows[at:at + b - a])
            at += b - a
    run([(0, 0, 10)])
    run([(5, 0, 7), (0, 10, 11)])
    run([(0, 11, 24), (5, 7, 24)])
    for s in got:
        assert U.error(np.concatenate(got[s]), want) < U.limit(f32), s
    hip.free_run_state(C.byref(state))
    hip.free_kv_cache_manager(C.byref(mgr))
    hip.nvllm_free_model(C.byref(weights))


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
    the previous one is collected, and without; tokens as the oracle's as long as its choice is not a near tie.  A second
    round of requests takes the slots of the first."""
    if stepwise:
        monkeypatch.setenv("NVLLM_ENGINE_STEPWISE", "1")
    path, cfg, w = U.model(tmp_path, "odd", seed=12)
    n_new = 14
    hip.nvllm_set_compute_dtype(capi.COMPUTE_F32 if f32 else capi.COMPUTE_BF16)
    for mode in (1, 0):
        hip.nvllm_set_logits_mode(mode)
        eng = capi.Engine(hip, path, 3, chunk_size=chunk, temperature=0.0, max_seq_len=64, recycle_blocks=1, max_steps=1 << 30)
        for again in range(2):
            prompts = [U.tokens(n, cfg["vocab"], 50 + n + again) for n in (1, 19, 40)]
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
    path, cfg, w = U.model(tmp_path, "odd", seed=12)
    hip.nvllm_set_compute_dtype(capi.COMPUTE_F32)
    hip.nvllm_set_logits_mode(1)
    runs = []
    for temp in (1e-3, 1.0, 1.0):
        eng = capi.Engine(hip, path, 1, temperature=temp, topp=0.9, seed=7, max_seq_len=64)
        eng.set_request(0, U.tokens(20, cfg["vocab"], 1), 10)
        eng.run_all()
        runs.append(eng.history(0).tolist())
        eng.close()
    hip.nvllm_set_logits_mode(0)
    want, margins = greedy(cfg, w, U.tokens(20, cfg["vocab"], 1), 10)
    if min(margins) > 0.02:
        assert runs[0] == want
    assert runs[1] == runs[2]


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


def test_generating_from_the_command_line(tmp_path):
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    path, cfg, w = U.model(tmp_path, "parts", seed=4)
    prompt = U.tokens(11, cfg["vocab"], 3).tolist()
    r = subprocess.run([os.path.join(root, "bin", "generate"), "--model", path, "-n", "6", "--prompt=" + ",".join(map(str, prompt)), "--dtype", "float32"],
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    new = [int(t) for t in r.stdout.split("|")[1].split(",")]
    want, margins = greedy(cfg, w, prompt, 6)
    assert new == want[len(prompt):] or min(margins) < 1e-4


@pytest.mark.parametrize("what", ["mixer", "heads", "experts", "decay", "weights_of"])
def test_a_folder_that_does_not_fit_is_refused(tmp_path, what):
    """Configurations the library does not know, or that the tensors contradict, end with a message and an error status."""
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    path, cfg, _ = U.model(tmp_path, "parts", seed=4)
    cfg = json.loads(json.dumps(cfg))
    lightning, window = cfg["layers"][0], cfg["layers"][1]
    if what == "mixer":
        window["type"] = "something_else"
    elif what == "heads":
        window["mixer"]["kv_heads"] = 3
    elif what == "experts":
        window["mlp"]["router"]["experts"] += 1
    elif what == "decay":
        lightning["mixer"]["decay"].append(0.5)
    else:
        cfg["layers"][3]["weights_of"] = 3
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    r = subprocess.run([os.path.join(root, "bin", "generate"), "--model", path, "-n", "1"], capture_output=True, text=True, timeout=100)
    assert r.returncode != 0 and r.stdout == ""
    assert {"mixer": "something_else", "heads": "inconsistent", "experts": "no tensor", "decay": "decay", "weights_of": "weights_of"}[what] in r.stderr
