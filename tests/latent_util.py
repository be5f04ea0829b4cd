"""Small configurations of the Suselorn design and helpers to run them through the library, for the tests."""
import numpy as np

from nvllm_amd import capi, synth
from tests import latent_oracle as O

M = synth.latent_mixer
# Sizes that no tile, page or wave likes; every list names what it is there for.
CONFIGS = {
    # widths off every multiple of 32, five heads, a loop in the middle, three streams
    "odd": synth.latent_config(72, 203, [(M(5, 20, 12, 28, 40, 36), 52), (M(5, 20, 12, 28, 40, 36), 44), (M(5, 20, 12, 28, 40, 36), 52)],
                               streams=3, loop=(1, 2, 3), softcap=7.5, eps=1e-3),
    # layers that differ from each other, one without a feed-forward, no loop, one stream
    "mixed": synth.latent_config(96, 320, [(M(4, 32, 16, 16, 64, 32), 64), (M(3, 48, 32, 40, 96, 64, base=500.0), None), (M(6, 16, 8, 24, 48, 96), 128)],
                                 streams=1),
    # more streams than the projection epilogue holds; the whole stack repeated; a wide latent
    "streams5": synth.latent_config(64, 150, [(M(2, 24, 16, 32, 160, 48), None), (M(2, 24, 16, 32, 160, 48), 80)], streams=5, loop=(0, 2, 2)),
    # one head, four streams, the loop at the end, rank and rotated part of real models
    "wide": synth.latent_config(128, 257, [(M(1, 64, 64, 64, 512, 96), 96), (M(20, 32, 64, 32, 512, 64, scale=0.09), 160)], streams=4, loop=(1, 2, 2)),
    # equal to none of its neighbours: 33 heads (two head groups), one of everything else
    "heads33": synth.latent_config(64, 130, [(M(33, 8, 4, 12, 24, 16), 40)], streams=2, loop=(0, 1, 1)),
}


def model(tmp, name, seed=3, edit=None, cfg=None):
    cfg = cfg or CONFIGS[name]
    path = str(tmp / f"{name}_{seed}")
    return path, cfg, synth.write_model_dir(path, cfg, seed=seed, edit=edit)


def engine(hip, path, f32, slots=4, tokens=2048, **kw):
    hip.nvllm_set_compute_dtype(capi.COMPUTE_F32 if f32 else capi.COMPUTE_BF16)
    hip.nvllm_set_logits_mode(0)
    return capi.Engine(hip, path, slots, num_blocks=-(-tokens // 16), max_seq_len=tokens, max_steps=1 << 30, **kw)


def error(got, want):
    """Worst row of: rms difference (mean taken off) over the rms of all wanted logits."""
    d = np.asarray(got, np.float64) - want
    d = d - d.mean(-1, keepdims=True)
    return float(np.sqrt((d * d).mean(-1)).max() / np.sqrt((want * want).mean()))


def limit(f32):
    return 3e-5 if f32 else 0.06


def tokens(n, vocab, seed):
    return np.random.Generator(np.random.PCG64(seed)).integers(0, vocab, n).astype(np.int32)


def feed_all(eng, plan, seqs):
    """plan: list of steps, each a list of (request, count).  Requests take a slot at their first portion and give it
    back with their last token.  Returns per request the logits of all its tokens."""
    at, slot, out = {}, {}, {r: [] for r in seqs}
    free = list(range(eng.n_seqs))[::-1]
    for step in plan:
        order = []
        for r, n in step:
            if r not in slot:
                slot[r], at[r] = free.pop(), 0
            eng.feed(slot[r], seqs[r][at[r]:at[r] + n], range(n))
            at[r] += n
            order.append((r, n))
        rows = eng.feed_run()
        i = 0
        for r, n in order:
            out[r].append(rows[i:i + n])
            i += n
            if at[r] == len(seqs[r]):
                eng.feed_end(slot[r])
                free.append(slot.pop(r))
    return {r: np.concatenate(v) for r, v in out.items()}


def oracle_logits(cfg, weights, seq):
    return O.forward(cfg, weights, seq)
