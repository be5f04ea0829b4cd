"""Every mechanism of the Suselorn design alone, through its operator entry point, against the plain restatement."""
import ctypes as C

import numpy as np
import pytest

from nvllm_amd import capi, synth
from tests import latent_oracle as O
from tests.util import f32

pytestmark = pytest.mark.gpu


def rng(seed):
    return np.random.Generator(np.random.PCG64(seed))


class Dev:
    """Device copies of arrays, freed together."""

    def __init__(self, lib):
        self.lib, self.held = lib, []

    def __call__(self, a):
        if a is None:
            return None
        p = self.lib.to_device(f32(a))
        self.held.append(p)
        return p

    def empty(self, n):
        p = self.lib.empty_device(4 * n)
        self.held.append(p)
        return p

    def close(self):
        for p in self.held:
            self.lib.free(p)


@pytest.mark.parametrize("streams,dim,T,bias,scale,norm", [(1, 7, 3, False, False, True), (2, 64, 33, True, True, True), (3, 50, 5, False, True, False),
                                                           (5, 96, 130, True, False, True), (9, 31, 2, True, True, True)])
def test_hyper_step(hip, streams, dim, T, bias, scale, norm):
    r = rng(streams)
    x, y = r.standard_normal((streams, T, dim)), r.standard_normal((T, dim))
    mix, out, w_in, alpha = r.standard_normal((streams, streams)), r.standard_normal(streams), r.standard_normal(streams), 0.7
    b, ls = r.standard_normal(dim) if bias else None, r.standard_normal(dim) if scale else None
    nw, nb = (r.standard_normal(dim), r.standard_normal(dim)) if norm else (None, None)
    want_y = (y + (0 if b is None else b)) * (1 if ls is None else ls)
    want_x = O.hyper_write(x, mix, out, want_y)
    u = O.hyper_read(want_x, w_in)
    want_z = O.dyt_norm(u, alpha, nw, nb) if norm else u
    d = Dev(hip)
    dx, dz = d(x.transpose(1, 0, 2)), d.empty(T * dim)
    hip.nvllm_hyper_step(dx, d(y), d(b), d(ls), d(np.concatenate([mix.ravel(), out, w_in, [alpha]])), d(nw), d(nb), dz, streams, dim, T)
    np.testing.assert_allclose(hip.to_host(dx, (T, streams, dim)), want_x.transpose(1, 0, 2), rtol=2e-5, atol=2e-5)
    np.testing.assert_allclose(hip.to_host(dz, (T, dim)), want_z, rtol=2e-5, atol=2e-5)
    # without a sublayer result the streams stay as they are
    dx = d(x.transpose(1, 0, 2))
    hip.nvllm_hyper_step(dx, None, None, None, d(np.concatenate([mix.ravel(), out, w_in, [alpha]])), d(nw), d(nb), dz, streams, dim, T)
    np.testing.assert_array_equal(hip.to_host(dx, (T, streams, dim)), f32(x.transpose(1, 0, 2)))
    u = O.hyper_read(x, w_in)
    np.testing.assert_allclose(hip.to_host(dz, (T, dim)), O.dyt_norm(u, alpha, nw, nb) if norm else u, rtol=2e-5, atol=2e-5)
    d.close()


def test_dynamic_tanh_alone(hip):
    """One stream with weight one: the norm by itself, also far outside tanh's linear range."""
    r = rng(0)
    T, dim = 5, 40
    x, w, b, alpha = r.standard_normal((T, dim)) * 30, r.standard_normal(dim), r.standard_normal(dim), -0.55
    d = Dev(hip)
    dz = d.empty(T * dim)
    hip.nvllm_hyper_step(d(x), None, None, None, d([1.0, 0.0, 1.0, alpha]), d(w), d(b), dz, 1, dim, T)
    np.testing.assert_allclose(hip.to_host(dz, (T, dim)), O.dyt_norm(x, alpha, w, b), rtol=1e-5, atol=1e-5)
    d.close()


def test_biased_swiglu_and_softcap(hip):
    r = rng(1)
    T, F = 7, 45
    g, u, bg, bu = (r.standard_normal(s) * 3 for s in ((T, F), (T, F), F, F))
    d = Dev(hip)
    o = d.empty(T * F)
    hip.nvllm_swiglu_bias(o, d(g), d(u), d(bg), d(bu), F, T)
    z = g + bg
    np.testing.assert_allclose(hip.to_host(o, (T, F)), z / (1 + np.exp(-z)) * (u + bu), rtol=1e-5, atol=1e-5)
    x = r.standard_normal(1000) * 40
    dx = d(x)
    hip.nvllm_softcap(dx, 12.5, 1000)
    np.testing.assert_allclose(hip.to_host(dx, (1000,)), O.softcap(x, 12.5), rtol=1e-5, atol=1e-5)
    d.close()


# ------------------------------------------------------------------ cached latents
class LatentPool:
    """A pool of cached latent rows with block tables, through the operator entry points."""

    def __init__(self, hip, rank, rot, elem, block_size=16, num_blocks=64):
        self.hip, self.rank, self.rot, self.elem = hip, rank, rot, elem
        self.mgr = capi.KVCacheManager()
        self.nb, self.bs = num_blocks, block_size
        hip.nvllm_latent_pool_init(C.byref(self.mgr), block_size, num_blocks, rank, rot, elem)
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

    def write(self, seq_ids, pos, kv, gain, eps, base):
        d = Dev(self.hip)
        self.hip.nvllm_latent_cache_write(C.byref(self.mgr), self.ptrs(), capi.ints(seq_ids), capi.ints(pos), d(kv), d(gain), eps, base, self.rank,
                                          self.rot, self.elem, len(pos))
        self.hip.device_sync()
        d.close()

    def attend(self, seq_ids, pos, q, sink, scale):
        T, H = q.shape[:2]
        d = Dev(self.hip)
        out = d.empty(T * H * self.rank)
        self.hip.nvllm_latent_attention(out, d(q), C.byref(self.mgr), self.ptrs(), capi.ints(seq_ids), capi.ints(pos), d(sink), scale, H, self.rank,
                                        self.rot, self.elem, T)
        res = self.hip.to_host(out, (T, H, self.rank))
        d.close()
        return res

    def rows(self):
        """[num_blocks * block_size, rank + rot] as fp32."""
        n = self.nb * self.bs
        if self.elem == 4:
            return self.hip.to_host(self.mgr.pool_k, (n, self.rank + self.rot))
        pad = lambda v: -(-v // 32) * 32
        row = pad(self.rank) + pad(self.rot)
        raw = synth.from_bf16(self.hip.to_host(self.mgr.pool_k, (n // 16, 16 * row), np.uint16))
        key, d = np.arange(16)[:, None], np.arange(row)[None, :]
        logical = raw[:, (d >> 5) * 512 + (key + 16 * ((d >> 3) & 3)) * 8 + (d & 7)].reshape(n, row)
        assert not logical[:, self.rank:pad(self.rank)].any() and not logical[:, pad(self.rank) + self.rot:].any(), "padding is not zero"
        return np.concatenate([logical[:, :self.rank], logical[:, pad(self.rank):pad(self.rank) + self.rot]], 1)

    def close(self):
        self.hip.free_kv_cache_manager(C.byref(self.mgr))


def rounded(a, elem):
    return f32(a).astype(np.float64) if elem == 4 else synth.from_bf16(synth.to_bf16(f32(a))).astype(np.float64)


@pytest.mark.parametrize("elem", [4, 2])
@pytest.mark.parametrize("rank,rot,bs", [(64, 32, 16), (40, 12, 16), (33, 2, 32), (512, 64, 16), (130, 40, 64), (16, 96, 48)])
def test_latent_rows_in_the_cache(hip, rank, rot, bs, elem):
    """Norm, rotation and placement of rows: late positions, blocks out of order, and rows nobody wrote stay zero."""
    r = rng(rank)
    pool = LatentPool(hip, rank, rot, elem, bs, 8)
    a, b = pool.sequence([5, 0, 3]), pool.sequence([7, 2])
    pos = [0, 1, bs - 1, bs, 2 * bs, 3 * bs - 1] + [0, bs + 3]
    seq = [a] * 6 + [b] * 2
    kv, gain, eps, base = r.standard_normal((8, rank + rot)) * 3, r.standard_normal(rank), 0.3, 700.0
    pool.write(seq, pos, kv, gain, eps, base)
    want = np.concatenate([O.rms_norm(kv[:, :rank], gain, eps), O.rotate_pairs(kv[:, rank:], np.array(pos), base, rot)], 1)
    rows = pool.rows()
    at = [pool.tables[s][1][p // bs] * bs + p % bs for s, p in zip(seq, pos)]
    tol = 2e-5 if elem == 4 else 2.0 ** -8
    np.testing.assert_allclose(rows[at], want, rtol=tol, atol=2e-5)
    rest = np.ones(len(rows), bool)
    rest[at] = False
    assert not rows[rest].any()
    pool.close()


def reference_attention(rows_of, q, pos, seq, sink, scale, rank):
    out = np.zeros((len(pos), q.shape[1], rank))
    for t, (s, p) in enumerate(zip(seq, pos)):
        k = rows_of[s][:p + 1]
        out[t] = np.stack([O.sink_softmax(scale * (q[t, h] @ k.T), sink[h]) @ k[:, :rank] for h in range(q.shape[1])])
    return out


def filled_pool(hip, rank, rot, elem, bs, lengths, seed):
    """A pool whose sequences hold `lengths` rows, written through the operator; blocks dealt in a shuffled order."""
    r = rng(seed)
    need = [-(-n // bs) for n in lengths]
    order = r.permutation(sum(need) + 3).tolist()
    pool = LatentPool(hip, rank, rot, elem, bs, sum(need) + 3)
    rows_of = []
    gain = np.ones(rank)
    for n, k in zip(lengths, need):
        s = pool.sequence([order.pop() for _ in range(k)])
        kv = r.standard_normal((n, rank + rot))
        pool.write([s] * n, list(range(n)), kv, gain, 1e-6, 100.0)
        at = np.array([pool.tables[s][1][p // bs] * bs + p % bs for p in range(n)])
        rows_of.append(pool.rows()[at].astype(np.float64))
    return pool, rows_of


# rank, rot, heads, block size: every register class of the tiled kernel, exact and not, one and several head groups,
# rows too wide for it, a block of three pages
SHAPES = [(64, 32, 6, 16), (16, 2, 1, 16), (40, 12, 5, 32), (96, 64, 16, 16), (128, 64, 12, 64), (200, 48, 3, 16), (256, 64, 20, 16), (320, 64, 2, 16),
          (512, 64, 32, 16), (512, 64, 33, 32), (576, 64, 2, 16), (64, 128, 3, 16), (48, 16, 7, 48)]


@pytest.mark.parametrize("elem", [4, 2])
@pytest.mark.parametrize("rank,rot,heads,bs", SHAPES)
def test_latent_attention_of_a_ragged_batch(hip, rank, rot, heads, bs, elem):
    """Decode rows beside prompt portions: lengths around page, block and 64-key borders, one long context."""
    lengths = [1, 15, 16, 17, 63, 64, 65, 129, 700]
    pool, rows_of = filled_pool(hip, rank, rot, elem, bs, lengths, rank + heads)
    r = rng(7)
    seq, pos = [], []
    for s, n in enumerate(lengths):
        span = {3: 17, 7: 2, 6: 40, 8: 35}.get(s, 1)     # whole prompt, two tokens, longer than one run, a portion of a long one
        first = {6: 20}.get(s, n - span)
        for p in range(first, first + span):
            seq.append(s)
            pos.append(p)
    q = rounded(r.standard_normal((len(pos), heads, rank + rot)), elem)
    sink = rounded(r.standard_normal(heads) * 2, 4)
    scale = 2.0 * (rank + rot) ** -0.5
    got = pool.attend(seq, pos, q, sink, scale)
    want = reference_attention(rows_of, q, pos, seq, sink, scale, rank)
    tol = 2e-5 if elem == 4 else 8e-3
    assert np.abs(got - want).max() < tol * np.abs(want).max() * 1.5, np.abs(got - want).max() / np.abs(want).max()
    pool.close()


@pytest.mark.parametrize("elem", [4, 2])
@pytest.mark.parametrize("decode", [True, False])
def test_one_far_key_and_nothing_beyond_the_token(hip, elem, decode):
    """One key stands out by far: wherever it lies -- first token, either side of a page's, a 64-key block's or a slice's
    border, the token itself -- it is found; one place beyond the token it is not seen at all."""
    rank, rot, heads, n = 64, 32, 6, 900
    pool, rows_of = filled_pool(hip, rank, rot, elem, 16, [n], 3)
    rows = rows_of[0]
    places = [0, 1, 15, 16, 17, 31, 32, 63, 64, 65, 127, 128, 255, 256, 257, 447, 448, 639, 640, 700]
    p = 700
    T = 1 if decode else 24
    sink = np.full(heads, -3.0)
    for k in places + [701]:
        pos = list(range(p - T + 1, p + 1))
        q = np.zeros((T, heads, rank + rot))
        q[:] = rounded(rows[k] / np.linalg.norm(rows[k]), elem)
        scale = 12.0
        got = pool.attend([0] * T, pos, q, sink, scale)
        want = reference_attention([rows], q, pos, [0] * T, sink, scale, rank)
        assert np.abs(got - want).max() < (3e-5 if elem == 4 else 1.5e-2) * np.abs(rows).max(), k
        near = np.abs(got[-1, 0] - rows[k, :rank]).max() < 0.05 * np.abs(rows[k, :rank]).max()
        assert near == (k <= p), k
    pool.close()


@pytest.mark.parametrize("elem", [4, 2])
def test_sink_takes_its_share(hip, elem):
    """A dominant sink empties the result, a negligible one leaves it, and one of a score's size halves a lone token's."""
    rank, rot, heads = 64, 32, 3
    pool, rows_of = filled_pool(hip, rank, rot, elem, 16, [300], 4)
    row = rows_of[0]
    q = rounded(rng(5).standard_normal((1, heads, rank + rot)) * 0.3, elem)
    s0 = float(q[0, 0] @ row[0])
    sink = np.array([s0, -60.0, 60.0])
    got = pool.attend([0], [0], q, sink, 1.0)[0]
    np.testing.assert_allclose(got[0], row[0, :rank] / 2, rtol=1e-2, atol=1e-2)
    np.testing.assert_allclose(got[1], row[0, :rank], rtol=1e-2, atol=1e-2)
    assert np.abs(got[2]).max() < 1e-12
    got = pool.attend([0], [299], q, np.array([2.0, 8.0, -1.0]), 1.0)
    want = reference_attention([row], q, [299], [0], [2.0, 8.0, -1.0], 1.0, rank)
    np.testing.assert_allclose(got, want, atol=(2e-5 if elem == 4 else 5e-3) * np.abs(want).max() + 1e-6)
    pool.close()


def test_slices_of_pages_and_one_slice_agree(hip):
    """A lone long sequence is cut into slices whose partial results are merged; many of them are not: same rows, same result."""
    rank, rot, heads, n = 64, 32, 5, 1500
    pool, _ = filled_pool(hip, rank, rot, 2, 16, [n], 9)
    q = rounded(rng(2).standard_normal((1, heads, rank + rot)), 2)
    sink = np.zeros(heads)
    one = pool.attend([0], [n - 1], q, sink, 0.2)
    for _ in range(599):
        pool.tables.append(pool.tables[0])
    many = pool.attend(list(range(600)), [n - 1] * 600, np.repeat(q, 600, 0), sink, 0.2)
    assert np.abs(many - many[:1]).max() == 0
    np.testing.assert_allclose(many[0], one[0], atol=6e-3 * np.abs(one).max())
    pool.close()
