"""Small configurations of the Simivik design and helpers to run them through the library, for the tests."""
import numpy as np

from nvllm_amd import synth
from tests import hybrid_oracle as O
from tests.latent_util import engine, error, feed_all, limit, tokens  # noqa: F401  (the same for every folder model)

L, A, E = synth.lightning_mixer, synth.window_mixer, synth.expert_mlp
# Sizes that no tile, page or wave likes; every list names what it is there for.
CONFIGS = {
    # both mixers, dense and experts, a borrowed layer of each kind; widths off every multiple of 32 and of 8
    "odd": synth.hybrid_config(75, 203, [(A(6, 2, 22, 13, size=19, keep_first=3, taps=3, rot=10, base=300.0, scale=0.3, softcap=9.0), E(21, 5, 2, 37)),
                                         (L(3, 20, 26), 51), 0, 1], eps=1e-3),
    # heads of 16-byte pieces with part of them turning; more than one expert per token, none shared; a layer without feed-forward
    "parts": synth.hybrid_config(96, 160, [(L(2, 64, 96), None), (A(4, 4, 48, 40, size=33, keep_first=17, taps=2, rot=16, base=50.0), E(64, 6, 3)),
                                           (A(8, 2, 32, 64, size=16, keep_first=0, taps=5, softcap=50.0), 96), 0]),
    # one token per window besides the kept ones; no convolution and no cap; wide heads; decays of 1 and 0
    "edges": synth.hybrid_config(64, 130, [(A(3, 1, 80, 160, size=1, keep_first=16, taps=None, rot=80, softcap=None), 40),
                                           (L(4, 130, 70, decay=[1.0, 0.0, 0.5, 0.999]), E(32, 4, 4, 32)), (A(2, 1, 32, 32, size=40, keep_first=1, taps=1), 33)]),
    # many heads of one group, a window wider than the tests' contexts, one expert of one
    "groups": synth.hybrid_config(64, 150, [(A(20, 1, 16, 16, size=5000, keep_first=2, taps=4, rot=4), E(16, 1, 1, 48)), (L(1, 32, 200), 64), 1]),
}


def model(tmp, name, seed=3, edit=None, cfg=None):
    cfg = cfg or CONFIGS[name]
    path = str(tmp / f"{name}_{seed}")
    return path, cfg, synth.write_model_dir(path, cfg, seed=seed, edit=edit)
