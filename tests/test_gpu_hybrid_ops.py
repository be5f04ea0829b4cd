"""Every mechanism of the Simivik design alone, through its operator entry point, against the plain restatement."""
import ctypes as C

import numpy as np
import pytest

from nvllm_amd import capi, synth
from tests import hybrid_oracle as O
from tests.test_gpu_latent_ops import Dev, rng, rounded

pytestmark = pytest.mark.gpu
BOTH = pytest.mark.parametrize("elem", [4, 2], ids=["fp32", "bf16"])


def pad32(n):
    return -(-n // 32) * 32


class WindowPool:
    """A pool of keys and values with block tables, through the operator entry points."""

    def __init__(self, hip, G, dim, vdim, elem, block_size=16, num_blocks=64):
        self.hip, self.G, self.dim, self.vdim, self.elem = hip, G, dim, vdim, elem
        self.mgr, self.nb, self.bs = capi.KVCacheManager(), num_blocks, block_size
        hip.nvllm_window_pool_init(C.byref(self.mgr), block_size, num_blocks, G, dim, vdim, elem)
        self.tables = []

    def sequence(self, blocks):
        arr = (C.c_int * len(blocks))(*blocks)
        self.tables.append((capi.BlockTable(C.cast(arr, capi.c_int_p), len(blocks)), arr))
        return len(self.tables) - 1

    def ptrs(self):
        p = (C.POINTER(capi.BlockTable) * len(self.tables))()
        for i, (bt, _) in enumerate(self.tables):
            p[i] = C.pointer(bt)
        return p

    def conv(self, seq_ids, pos, raw, H, taps=None, state=None, base=100.0, rot=0):
        """raw [T, channels] -> queries [T, H, dim]; keys and values go to the pool.  taps [channels, n]."""
        d, T = Dev(self.hip), len(pos)
        q = d.empty(T * H * self.dim)
        self.hip.nvllm_conv_rope(q, d(raw), None if taps is None else d(np.ascontiguousarray(taps.T)), 1 if taps is None else taps.shape[1], state,
                                 C.byref(self.mgr), self.ptrs(), capi.ints(seq_ids), capi.ints(pos), base, rot, H, self.G, self.dim, self.vdim, self.elem, T)
        out = self.hip.to_host(q, (T, H, self.dim))
        d.close()
        return out

    def write(self, seq, keys, values):
        n = len(keys)
        raw = np.concatenate([np.zeros((n, self.dim * self.G)), keys.reshape(n, -1), values.reshape(n, -1)], 1)
        self.conv([seq] * n, list(range(n)), raw, self.G)

    def attend(self, seq_ids, pos, q, scale, cap, size, keep):
        (T, H), d = q.shape[:2], Dev(self.hip)
        out = d.empty(T * H * self.vdim)
        self.hip.nvllm_window_attention(out, d(q), C.byref(self.mgr), self.ptrs(), capi.ints(seq_ids), capi.ints(pos), scale, cap, size, keep, H, self.G,
                                        self.dim, self.vdim, self.elem, T)
        res = self.hip.to_host(out, (T, H, self.vdim))
        d.close()
        return res

    def rows(self, seq, n):
        """Keys [n, G, dim] and values [n, G, vdim] of a sequence as they lie in the pool; the padding must be zero."""
        total = self.nb * self.bs
        at = np.array([self.tables[seq][1][p // self.bs] * self.bs + p % self.bs for p in range(n)])
        kl, vl = (self.dim, self.vdim) if self.elem == 4 else (pad32(self.dim), pad32(self.vdim))
        raw = self.hip.to_host(self.mgr.pool_k, (total * self.G * (kl + vl),), np.float32 if self.elem == 4 else np.uint16)
        raw = raw if self.elem == 4 else synth.from_bf16(raw)
        k, v = raw[:total * self.G * kl], raw[total * self.G * kl:]
        if self.elem == 4:
            return k.reshape(total, self.G, kl)[at], v.reshape(total, self.G, vl)[at]
        key, d = np.arange(16)[:, None], np.arange(kl)[None, :]
        k = k.reshape(total // 16, self.G, 16 * kl)[:, :, (d >> 5) * 512 + (key + 16 * ((d >> 3) & 3)) * 8 + (d & 7)]
        d = np.arange(vl)[None, :]
        v = v.reshape(total // 16, self.G, 16 * vl)[:, :, (d >> 4) * 256 + ((key >> 2) * 16 + (d & 15)) * 4 + (key & 3)]
        k, v = k.transpose(0, 2, 1, 3).reshape(total, self.G, kl)[at], v.transpose(0, 2, 1, 3).reshape(total, self.G, vl)[at]
        assert not k[..., self.dim:].any() and not v[..., self.vdim:].any(), "padding is not zero"
        return k[..., :self.dim], v[..., :self.vdim]

    def close(self):
        self.hip.free_kv_cache_manager(C.byref(self.mgr))


# ------------------------------------------------------------------ convolution, rotation, cache
@BOTH
@pytest.mark.parametrize("H,G,dim,vdim,taps,rot,bs", [(2, 1, 64, 32, 4, 64, 16), (6, 2, 22, 13, 3, 10, 32), (4, 4, 48, 40, 2, 16, 16), (1, 1, 8, 8, 1, 0, 16),
                                                      (3, 1, 80, 160, 5, 48, 64), (2, 2, 32, 24, 9, 4, 16), (5, 1, 6, 7, None, 6, 16)])
def test_convolution_rotation_and_cache(hip, H, G, dim, vdim, taps, rot, bs, elem):
    """Two sequences in portions down to one token, side by side, after another sequence has used slot and blocks: the
    convolution goes on where the last portion ended, and starts from zeros at position 0."""
    r = rng(dim + vdim)
    channels, n, base = H * dim + G * (dim + vdim), [61, 40], 77.0
    w = None if taps is None else np.asarray(r.standard_normal((channels, taps)), np.float32).astype(np.float64)
    pool = WindowPool(hip, G, dim, vdim, elem, bs, 24)
    per = -(-64 // bs)
    seqs = [pool.sequence(list(range(i * per, (i + 1) * per))[::-1]) for i in range(2)]
    u = [rounded(r.standard_normal((k, channels)) * 2, elem) for k in n]
    state = hip.to_device(np.zeros(2 * max((taps or 1) - 1, 1) * channels, np.float32))
    for first in (True, False):
        if first:   # what slots and blocks held before
            pool.conv([0] * 7 + [1] * 3, list(range(7)) + list(range(3)), r.standard_normal((10, channels)) * 9, H, w, state, base, rot)
            continue
        got = [[], []]
        cuts = [[1, 2, 17, 1, 3, 16, 1, 4, 2, 14], [5, 1, 1, 2, 1, 30]]
        at = [0, 0]
        for step in range(10):
            ids, pos, raw = [], [], []
            for s in seqs:
                k = cuts[s][step] if step < len(cuts[s]) else 0
                ids += [s] * k
                pos += list(range(at[s], at[s] + k))
                raw.append(u[s][at[s]:at[s] + k])
                at[s] += k
            q = pool.conv(ids, pos, np.concatenate(raw), H, w, state, base, rot)
            for s in seqs:
                got[s].append(q[[i for i, x in enumerate(ids) if x == s]])
        assert at == n
    tol = 2e-5 if elem == 4 else 2.0 ** -7
    for s in seqs:
        y = u[s] if w is None else O.causal_conv(u[s], w)
        q, k, v = np.split(y, [H * dim, (H + G) * dim], axis=1)
        q, k, v = q.reshape(n[s], H, dim), k.reshape(n[s], G, dim), v.reshape(n[s], G, vdim)
        if rot:
            q, k = (O.rotate_half(z, np.arange(n[s]), base, rot) for z in (q, k))
        have_k, have_v = pool.rows(s, n[s])
        for have, want in ((np.concatenate(got[s]), q), (have_k, k), (have_v, v)):
            np.testing.assert_allclose(have, want, rtol=tol, atol=tol * 0.2)
    hip.free(state)
    pool.close()


@pytest.mark.parametrize("H,G,dim,vdim,cuts", [(4, 2, 32, 32, [[257, 300], [1, 90], [40]]), (96, 96, 128, 128, [[301, 1], [402, 7], [200, 95]])])
def test_convolution_of_large_batches(hip, H, G, dim, vdim, cuts):
    """Batches large enough for threads that walk two and four tokens: portions that start anywhere among them."""
    r = rng(H)
    channels, taps, base = H * dim + G * (dim + vdim), 4, 500.0
    w = np.asarray(r.standard_normal((channels, taps)), np.float32).astype(np.float64)
    pool = WindowPool(hip, G, dim, vdim, 2, 16, 150)
    seqs = [pool.sequence(list(range(50 * i, 50 * i + 50))) for i in range(3)]
    u = [rounded(r.standard_normal((sum(c), channels)), 2) for c in cuts]
    state = hip.to_device(np.zeros(3 * 3 * channels, np.uint16))
    at, got = [0, 0, 0], [[], [], []]
    for step in range(2):
        ids, pos, raw = [], [], []
        for s in (1, 0, 2):
            k = cuts[s][step] if step < len(cuts[s]) else 0
            ids += [s] * k
            pos += list(range(at[s], at[s] + k))
            raw.append(u[s][at[s]:at[s] + k])
            at[s] += k
        q = pool.conv(ids, pos, np.concatenate(raw), H, w, state, base, dim)
        for s in seqs:
            got[s].append(q[[i for i, x in enumerate(ids) if x == s]])
    for s in seqs:
        n = len(u[s])
        q, k, v = np.split(O.causal_conv(u[s], w), [H * dim, (H + G) * dim], axis=1)
        q, k = (O.rotate_half(z.reshape(n, -1, dim), np.arange(n), base, dim) for z in (q, k))
        have_k, have_v = pool.rows(s, n)
        for have, want in ((np.concatenate(got[s]), q), (have_k, k), (have_v, v.reshape(n, G, vdim))):
            np.testing.assert_allclose(have, want, rtol=2.0 ** -7, atol=2e-3)
    hip.free(state)
    pool.close()


# ------------------------------------------------------------------ attention
def filled(hip, G, dim, vdim, elem, bs, lengths, seed, spread=1.0):
    r = rng(seed)
    need = [-(-n // bs) for n in lengths]
    order = r.permutation(sum(need) + 3).tolist()
    pool, kv = WindowPool(hip, G, dim, vdim, elem, bs, sum(need) + 3), []
    for n, k in zip(lengths, need):
        s = pool.sequence([order.pop() for _ in range(k)])
        kv.append((rounded(r.standard_normal((n, G, dim)) * spread, elem), rounded(r.standard_normal((n, G, vdim)), elem)))
        pool.write(s, *kv[-1])
    return pool, kv


def reference(kv, q, pos, seq, scale, cap, size, keep):
    out = []
    for t, (s, p) in enumerate(zip(seq, pos)):
        k, v = kv[s][0][:p + 1], kv[s][1][:p + 1]
        per = q.shape[1] // k.shape[1]
        seen = O.visible(p + 1, size, keep)[p]
        row = []
        for h in range(q.shape[1]):
            z = k[seen, h // per] @ q[t, h] * scale
            z = cap * np.tanh(z / cap) if cap else z
            e = np.exp(z - z.max())
            row.append(e / e.sum() @ v[seen, h // per])
        out.append(row)
    return np.array(out)


# heads, groups, dim, vdim, block size: every register class of the tiled kernel, exact and not; one and several heads per
# group, more than 16, none that divides the item; sizes too wide for it, a block of three pages
SHAPES = [(6, 2, 64, 64, 16), (4, 4, 16, 24, 32), (5, 1, 40, 80, 16), (8, 2, 128, 128, 64), (3, 1, 33, 112, 16), (3, 3, 192, 256, 16), (2, 1, 256, 64, 16),
          (2, 2, 256, 256, 32), (4, 1, 128, 64, 16), (33, 1, 32, 32, 16), (16, 1, 64, 48, 16), (2, 1, 300, 40, 16), (6, 2, 24, 24, 48)]
MASKS = [(70, 5, 28.0), (1, 0, 0.0), (33, 17, 60.0), (1 << 30, 0, 5.0), (16, 32, 0.0)]


@BOTH
@pytest.mark.parametrize("H,G,dim,vdim,bs", SHAPES)
def test_windowed_attention_of_a_ragged_batch(hip, H, G, dim, vdim, bs, elem):
    """Single tokens beside prompt portions: lengths around page and run borders, one long context, several masks and caps."""
    lengths = [1, 15, 16, 17, 63, 64, 65, 129, 700]
    pool, kv = filled(hip, G, dim, vdim, elem, bs, lengths, dim + H)
    r = rng(7)
    seq, pos = [], []
    for s, n in enumerate(lengths):
        span = {3: 17, 7: 2, 6: 40, 8: 135}.get(s, 1)     # whole prompt, two tokens, longer than an item, longer than a run
        first = {6: 20}.get(s, n - span)
        seq += [s] * span
        pos += list(range(first, first + span))
    q = rounded(r.standard_normal((len(pos), H, dim)), elem)
    for size, keep, cap in MASKS:
        got = pool.attend(seq, pos, q, 2.5 * dim ** -0.5, cap, size, keep)
        want = reference(kv, q, pos, seq, 2.5 * dim ** -0.5, cap, size, keep)
        worst = np.abs(got - want).max() / np.abs(want).max()
        assert worst < (2e-5 if elem == 4 else 8e-3) * 1.5, (size, keep, cap, worst)
    pool.close()


# batches large enough for items of two and four column groups: one head per group and several, exact sizes and not
@pytest.mark.parametrize("H,G,dim,vdim,tokens", [(32, 32, 64, 64, 2048), (32, 8, 64, 64, 2048), (32, 8, 40, 48, 2048), (32, 32, 64, 64, 1024), (24, 8, 64, 64, 1536), (24, 8, 48, 40, 1536),
                                                 (32, 32, 128, 128, 1024), (32, 16, 80, 112, 1024), (6, 2, 192, 160, 600)])
def test_windowed_attention_of_large_batches(hip, H, G, dim, vdim, tokens):
    n = tokens // 4
    pool, kv = filled(hip, G, dim, vdim, 2, 16, [n + 30] * 4, tokens + dim)
    r = rng(11)
    seq = np.repeat(np.arange(4), n)
    pos = np.concatenate([np.arange(n) + first for first in (0, 7, 16, 30)])
    q = rounded(r.standard_normal((tokens, H, dim)), 2)
    some = np.unique(np.concatenate([r.integers(0, tokens, 60), [0, n - 1, n, n + 1, tokens - 1]]))
    for size, keep, cap in ((50, 5, 27.0), (77, 0, 0.0), (16, 40, 45.0)):
        got = pool.attend(seq.tolist(), pos.tolist(), q, 2.5 * dim ** -0.5, cap, size, keep)
        want = reference(kv, q[some], pos[some], seq[some], 2.5 * dim ** -0.5, cap, size, keep)
        worst = np.abs(got[some] - want).max() / np.abs(want).max()
        assert np.isfinite(got).all() and worst < 1.2e-2, (size, keep, cap, worst)
    pool.close()


@BOTH
@pytest.mark.parametrize("decode", [True, False])
@pytest.mark.parametrize("size,keep", [(64, 4), (65, 16), (63, 17), (200, 1), (1, 33), (16, 0)])
def test_one_key_stands_out(hip, elem, decode, size, keep):
    """One key's score stands out: it decides where it is seen -- kept tokens, inside the window, the token itself -- and does
    not just outside: one before the window, one past the kept ones, one past the token; around page borders too."""
    H, G, dim, vdim, n, scale, cap = 4, 2, 64, 64, 420, 0.5, 25.0
    pool, kv = filled(hip, G, dim, vdim, elem, 16, [n], 3, spread=0.5)
    k, v = kv[0]
    T = 1 if decode else 24
    for p in (397, 400, 415, 407):
        edges = {0, 1, keep - 1, keep, keep + 1, 15, 16, 17, p - size, p - size + 1, p - size - 1, p - 1, p, p + 1, p - T + 1, p - T - size + 1, p - T - size + 2, 383, 384}
        for j in sorted(e for e in edges if 0 <= e < n):
            pos = list(range(p - T + 1, p + 1))
            q = np.zeros((T, H, dim))
            for h in range(H):
                q[:, h] = rounded(9.0 * k[j, h // 2] / np.linalg.norm(k[j, h // 2]), elem)
            got = pool.attend([0] * T, pos, q, scale, cap, size, keep)
            want = reference(kv, q, pos, [0] * T, scale, cap, size, keep)
            assert np.abs(got - want).max() < (4e-5 if elem == 4 else 2e-2) * np.abs(v).max(), (p, j)
            seen = j <= p and (p - j < size or j < keep)
            if size > 1:   # (alone in its window it would be exact)
                assert (np.abs(got[-1] - np.repeat(v[j], 2, 0)).max() < 0.6) == seen, (p, j)
    pool.close()


@pytest.mark.parametrize("cap", [0.0, 20.0, 60.0])
def test_slices_of_pages_and_one_slice_agree(hip, cap):
    """A lone long sequence is cut into slices whose partial results are merged; many of them are not: same rows, same result."""
    H, G, dim, vdim, n = 6, 2, 64, 88, 3000
    pool, kv = filled(hip, G, dim, vdim, 2, 16, [n], 9)
    q = rounded(rng(2).standard_normal((1, H, dim)), 2)
    one = pool.attend([0], [n - 1], q, 0.2, cap, 2900, 5)
    for _ in range(299):
        pool.tables.append(pool.tables[0])
    many = pool.attend(list(range(300)), [n - 1] * 300, np.repeat(q, 300, 0), 0.2, cap, 2900, 5)
    assert np.abs(many - many[:1]).max() == 0
    np.testing.assert_allclose(many[0], one[0], rtol=2.0 ** -7, atol=2e-3 * np.abs(one).max())   # (a step of bf16)
    np.testing.assert_allclose(one, reference(kv, q, [n - 1], [0], 0.2, cap, 2900, 5), atol=1e-2 * np.abs(one).max())
    pool.close()


@BOTH
def test_capped_scores_far_outside_the_cap(hip, elem):
    """Scores many times the cap, of either sign: weights stay finite and the cap decides."""
    pool, kv = filled(hip, 1, 32, 32, elem, 16, [90], 4, spread=6.0)
    q = rounded(rng(5).standard_normal((3, 2, 32)) * 20, elem)
    for cap in (2.0, 32.0, 33.0):
        got = pool.attend([0] * 3, [87, 88, 89], q, 1.0, cap, 50, 3)
        want = reference(kv, q, [87, 88, 89], [0] * 3, 1.0, cap, 50, 3)
        assert np.isfinite(got).all()
        np.testing.assert_allclose(got, want, atol=(5e-5 if elem == 4 else 1.2e-2) * np.abs(kv[0][1]).max())
    pool.close()


# ------------------------------------------------------------------ linear attention with decay
@BOTH
@pytest.mark.parametrize("H,dim,vdim", [(2, 32, 32), (3, 20, 26), (2, 64, 64), (1, 96, 48), (2, 128, 128), (1, 40, 200), (1, 256, 70), (2, 300, 16), (1, 130, 33)])
def test_linear_attention(hip, H, dim, vdim, elem):
    """Portions of many sizes beside single tokens; results and the 32-bit state against the plain recurrence; slots used before."""
    r = rng(dim * vdim)
    decay = np.array([0.6, 1.0, 0.97])[:H] if H > 1 else np.array([0.9])
    cuts = [[1] * 9 + [2, 3], [2, 64, 65, 1, 1, 63], [130, 1, 17, 2], [16, 15, 1, 200]]
    n = [sum(c) for c in cuts]
    data = [[rounded(r.standard_normal((k, H, w)) * 0.7, elem) for w in (dim, dim, vdim, vdim)] for k in n]
    gain = rounded(1 + 0.3 * r.standard_normal(H * vdim), 4)
    state = hip.to_device(np.asarray(r.standard_normal((4, H, dim, vdim)), np.float32))   # another sequence's remains
    d = Dev(hip)
    d_gain = d(gain)
    got, sums, at = [[] for _ in cuts], [[] for _ in cuts], [0] * 4
    for step in range(11):
        ids, pos, parts = [], [], []
        for s, c in enumerate(cuts):
            if step < len(c):
                ids += [s] * c[step]
                pos += list(range(at[s], at[s] + c[step]))
                parts.append([x[at[s]:at[s] + c[step]] for x in data[s]])
                at[s] += c[step]
        T = len(ids)
        q, k, v, g = (np.concatenate(x) for x in zip(*parts))
        e = Dev(hip)
        out, ss = e.empty(T * H * vdim), e.empty(T)
        hip.nvllm_lightning(out, ss if elem == 2 else None, e(q), e(k), e(v), e(g), d_gain, (C.c_float * H)(*decay), state, capi.ints(ids), capi.ints(pos), H, dim, vdim, elem, T)
        o, z = hip.to_host(out, (T, H, vdim)), hip.to_host(ss, (T,))
        e.close()
        for s in range(4):
            mine = [i for i, x in enumerate(ids) if x == s]
            got[s].append(o[mine])
            sums[s].append(z[mine])
    have = hip.to_host(state, (4, H, dim, vdim))
    exact = np.float32(decay).astype(np.float64)
    for s in range(4):
        q, k, v, g = data[s]
        o, st = O.decayed_state(q, k, v, exact)
        size = np.abs(o).max()
        assert np.abs(have[s] - st).max() < 4e-6 * np.abs(st).max(), s      # the state is of 32 bits in both forms
        if elem == 4:
            assert np.abs(np.concatenate(got[s]) - o).max() < 5e-6 * size, s
        else:
            want = o * gain.reshape(H, vdim) * O.sigmoid(g)
            np.testing.assert_allclose(np.concatenate(got[s]), want, rtol=2.0 ** -7, atol=2e-5 * size)
            np.testing.assert_allclose(np.concatenate(sums[s]), (o * o).sum((1, 2)), rtol=2e-5)
    d.close()
    hip.free(state)


def test_decays_of_nothing_and_of_everything(hip):
    """decay 0 remembers the token alone, decay 1 forgets nothing; a key far back is found by its direction."""
    H, dim, n = 2, 64, 500
    r = rng(3)
    k = rounded(r.standard_normal((n, H, dim)) * 0.002, 2)
    q, v = rounded(r.standard_normal((n, H, dim)) * 0.02, 2), rounded(r.standard_normal((n, H, dim)), 2)
    k[7] = 0
    k[7, :, 5] = 1.0
    q[-1] = 0
    q[-1, :, 5] = 1.0                      # asks for token 7
    d = Dev(hip)
    state, out = d.empty(H * dim * dim), d.empty(n * H * dim)
    ones = d(np.ones(H * dim))
    hip.nvllm_lightning(out, None, d(q), d(k), d(v), d(np.full((n, H, dim), 30.0)), ones, (C.c_float * 2)(0.0, 1.0), state, capi.ints([0] * n), capi.ints(range(n)), H,
                        dim, dim, 2, n)
    o = hip.to_host(out, (n, H, dim))
    want, _ = O.decayed_state(q, k, v, [0.0, 1.0])
    np.testing.assert_allclose(o, want, rtol=2.0 ** -7, atol=1e-4)
    assert np.abs(o[-1, 1] - v[7, 1]).max() < 0.3 and np.abs(o[-1, 0]).max() < 0.1
    d.close()


# ------------------------------------------------------------------ mixture of experts
@BOTH
@pytest.mark.parametrize("T,D,ff,E,top", [(1, 64, 32, 8, 2), (3, 40, 21, 5, 5), (70, 96, 64, 16, 1), (64, 64, 48, 3, 2), (300, 64, 32, 130, 3), (600, 72, 33, 4, 2),
                                          (257, 64, 160, 1, 1), (520, 64, 64, 6, 1)])
def test_experts(hip, T, D, ff, E, top, elem):
    """The chosen experts, their scores and the sum of what they give, from one token to hundreds per expert; some experts
    get nothing, one gets most."""
    r = rng(T + E)
    z = r.permuted(np.tile(np.linspace(-2.5, 2.0, E), (T, 1)), axis=1)
    if E > 2:
        z[:T * 2 // 3, 1] = 3.0            # a favourite
        z[:, E - 1] = -4.0                 # never chosen, unless all are
    x = rounded(r.standard_normal((T, D)), elem)
    gate, up = (rounded(r.standard_normal((E, ff, D)) * D ** -0.5, elem) for _ in range(2))
    down = rounded(r.standard_normal((E, D, ff)) * ff ** -0.5, elem)
    d = Dev(hip)
    out, choice, score = d.empty(T * D), d.empty(T * top), d.empty(T * top)
    hip.nvllm_expert_ff(out, choice, score, d(x), d(z), d(gate), d(up), d(down), D, ff, E, top, elem, T)
    chosen, weight = O.route(z, top)
    np.testing.assert_array_equal(hip.to_host(choice, (T, top), np.int32), chosen)
    np.testing.assert_allclose(hip.to_host(score, (T, top)), weight, rtol=1e-6)
    want = np.zeros((T, D))
    for t in range(T):
        for e, w in zip(chosen[t], weight[t]):
            want[t] += O.gated(w * x[t], gate[e], up[e], down[e])
    got = hip.to_host(out, (T, D))
    d.close()
    assert np.abs(got - want).max() < (1e-5 if elem == 4 else 1e-2) * np.abs(want).max()


def test_router_prefers_the_first_of_equals(hip):
    z = np.zeros((4, 70))
    z[1, 69] = z[1, 3] = 1.0
    z[2, 64:] = -1.0
    z[3] = -np.arange(70)
    d = Dev(hip)
    choice = d.empty(4 * 3)
    hip.nvllm_expert_ff(None, choice, None, None, d(z), None, None, None, 32, 32, 70, 3, 4, 4)
    np.testing.assert_array_equal(hip.to_host(choice, (4, 3), np.int32), [[0, 1, 2], [3, 69, 0], [0, 1, 2], [0, 1, 2]])
    d.close()
