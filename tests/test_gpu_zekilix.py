"""GPU checks of the Zekilix mechanisms, each alone through its operator entry point, against the plain
restatement in oracle/layered.py: hyper-connections (a launch of their own, and folded into a decode matmul), the
clamped gate and capped outputs of the matmuls, the matrix memory, attention whose values are its keys.  Whole
models of the design run in test_gpu_layered.py."""
import ctypes as C

import numpy as np
import pytest

from coeus_amd import _lib
from coeus_amd.device import DeviceArray
from coeus_amd.plugin import _check
from gpu_util import Weight, dev
from layered_util import bf16_round
from oracle import layered as L
from test_gpu_layered import off

pytestmark = pytest.mark.gpu


# ------------------------------------------------------------------ hyper-connections
class Hyper:
    """One step between two sublayers on random streams; parts can be left out."""

    def __init__(self, rows, hidden, streams, with_y=True, with_in=True, with_norm=True, seed=0, shift=0.0):
        rng = np.random.default_rng(seed + rows + hidden + streams)
        f = lambda a: np.asarray(a, np.float32)
        self.x, self.y = f(rng.normal(size=(rows, streams, hidden)) + shift), f(rng.normal(size=(rows, hidden)) * 3)
        self.mix, self.out = f(rng.normal(size=(streams, streams))), f(rng.uniform(-1.5, 1.5, streams))
        self.w_in, self.norm = f(rng.uniform(-1, 1, streams)), f(rng.uniform(0.5, 1.5, hidden))
        self.mult, self.eps = 0.37, 1e-3
        self.use = with_y, with_in, with_norm
        self.keep = [dev(a) for a in (self.y, self.mix, self.out, self.w_in, self.norm)]
        y, mix, out, w_in, norm = (k.ptr for k in self.keep)
        self.step = _lib.CHyperStep(streams, y if with_y else None, mix if with_y else None, out if with_y else None,
                                    w_in if with_in else None, norm if with_norm else None, self.mult, self.eps)

    def want(self):
        """(new streams, u), float64"""
        y, w_in, norm = self.use
        xs = np.moveaxis(self.x.astype(np.float64), 1, 0)
        if y:
            xs = L.hyper_write(xs, self.mix.astype(np.float64), self.out.astype(np.float64), self.y.astype(np.float64), self.mult)
        u = L.hyper_read(xs, self.w_in.astype(np.float64) if w_in else np.ones(len(xs)))
        return np.moveaxis(xs, 0, 1), L.layer_norm(u, self.norm.astype(np.float64), self.eps) if norm else u


@pytest.mark.parametrize("use", [(True, True, True), (False, True, True), (True, False, True), (True, False, False), (False, False, False)])
@pytest.mark.parametrize("rows,hidden,streams", [(1, 64, 1), (5, 130, 3), (3, 4096, 4), (2, 8196, 2), (300, 96, 8), (2, 36, 5), (4, 1000, 6),
                                                 (3, 7, 2), (2, 5000, 3)])
def test_hyper(rows, hidden, streams, use):
    t = Hyper(rows, hidden, streams, *use, shift=4.0)
    dx, du = dev(t.x), DeviceArray((rows, hidden))
    _check(_lib.load().coeus_op_hyper(C.byref(t.step), dx.ptr, rows, hidden, du.ptr, None))
    xs, u = t.want()
    assert off(dx.to_host(), xs) < 1e-6 and max(off(a, b) for a, b in zip(du.to_host(), u)) < 1e-5


def test_hyper_output_over_its_input():
    """u may take y's place."""
    t = Hyper(3, 200, 3)
    dx = dev(t.x)
    _check(_lib.load().coeus_op_hyper(C.byref(t.step), dx.ptr, 3, 200, t.keep[0].ptr, None))
    xs, u = t.want()
    assert off(dx.to_host(), xs) < 1e-6 and off(t.keep[0].to_host(), u) < 1e-5


@pytest.mark.parametrize("wd", [_lib.W_F32, _lib.W_BF16])
@pytest.mark.parametrize("with_y", [True, False])
@pytest.mark.parametrize("batch,k,n,streams", [(1, 96, 40, 3), (3, 58, 131, 2), (4, 128, 64, 4), (2, 1024, 300, 1), (1, 4096, 52, 4), (3, 250, 17, 3),
                                               (1, 2050, 34, 2), (2, 4000, 20, 4), (1, 6000, 18, 3), (1, 520, 8230, 4), (2, 64, 9001, 2)])
def test_hyper_gemv(wd, with_y, batch, k, n, streams):
    rng = np.random.default_rng(k + n)
    w = rng.normal(size=(k, n)).astype(np.float32) / np.float32(np.sqrt(k))
    t, W = Hyper(batch, k, streams, with_y, shift=2.0), Weight(wd, w)
    dx, new, y = dev(t.x), DeviceArray(t.x.shape).zero_(), DeviceArray((batch, n))
    _check(_lib.load().coeus_op_hyper_gemv(W.h, C.byref(t.step), dx.ptr, batch, new.ptr, 0, 0.0, y.ptr, None))
    xs, u = t.want()
    assert off(y.to_host(), u @ W.dequantize().astype(np.float64)) < 3e-6
    assert np.array_equal(dx.to_host(), t.x)
    assert off(new.to_host(), xs) < 1e-6 if with_y else not new.to_host().any()


def test_hyper_refusals():
    lib, t = _lib.load(), Hyper(2, 64, 3)
    dx, u = dev(t.x), DeviceArray((2, 64))
    t.step.streams = 9
    assert lib.coeus_op_hyper(C.byref(t.step), dx.ptr, 2, 64, u.ptr, None) == _lib.INVALID_INPUT
    t.step.streams = 3
    assert lib.coeus_op_hyper(C.byref(t.step), dx.ptr, 0, 64, u.ptr, None) == _lib.INVALID_INPUT
    W = Weight(_lib.W_F32, np.zeros((64, 8), np.float32))
    y = DeviceArray((2, 8))
    assert lib.coeus_op_hyper_gemv(W.h, C.byref(t.step), dx.ptr, 2, dx.ptr, 0, 0.0, y.ptr, None) == _lib.INVALID_INPUT  # in place
    assert lib.coeus_op_hyper_gemv(W.h, C.byref(t.step), dx.ptr, 5, u.ptr, 0, 0.0, y.ptr, None) == _lib.INVALID_INPUT
    t.step.streams = 5
    assert lib.coeus_op_hyper_gemv(W.h, C.byref(t.step), dx.ptr, 1, u.ptr, 0, 0.0, y.ptr, None) == _lib.INVALID_INPUT
    assert lib.coeus_op_matmul_limited(W.h, dx.ptr, 1, 0, _lib.EPI_CLAMP_GATE, 0.0, y.ptr, None) == _lib.INVALID_INPUT
    assert lib.coeus_op_matmul_limited(W.h, dx.ptr, 1, 0, _lib.EPI_SILU_GATE, 1.0, y.ptr, None) == _lib.INVALID_INPUT


# ------------------------------------------------------------------ epilogues with a limit
def clamped(z, limit):
    g, u = np.minimum(z[:, 0::2], limit), np.clip(z[:, 1::2], -limit, limit)
    return g * L.sigmoid(1.702 * g) * (u + 1.0)


@pytest.mark.parametrize("epi", [_lib.EPI_CLAMP_GATE, _lib.EPI_SOFTCAP, _lib.EPI_NONE])
@pytest.mark.parametrize("wd", [_lib.W_F32, _lib.W_BF16])
@pytest.mark.parametrize("rows,k,n,prompt", [(1, 96, 64, 0), (3, 130, 34, 0), (16, 64, 130, 0), (2, 2048, 512, 0), (1, 64, 130, 1),
                                             (5, 96, 34, 1), (70, 130, 200, 1), (150, 128, 512, 1), (600, 256, 1024, 1), (1100, 64, 2816, 1),
                                             (2048, 512, 2048, 1), (300, 1024, 384, 1)])
def test_limited_epilogues(epi, wd, rows, k, n, prompt):
    rng = np.random.default_rng(rows + n)
    x = bf16_round(rng.normal(size=(rows, k)))  # (a bf16 prompt matmul rounds its activations)
    W = Weight(wd, rng.normal(size=(k, n)).astype(np.float32) * np.float32(2.0 / np.sqrt(k)))
    z = x.astype(np.float64) @ W.dequantize().astype(np.float64)
    limit = 1.3
    want = {_lib.EPI_CLAMP_GATE: lambda: clamped(z, limit), _lib.EPI_SOFTCAP: lambda: L.soft_cap(z, limit), _lib.EPI_NONE: lambda: z}[epi]()
    dx, y = dev(x, np.float32), DeviceArray(want.shape)
    _check(_lib.load().coeus_op_matmul_limited(W.h, dx.ptr, rows, prompt, epi, limit, y.ptr, None))
    got = y.to_host()
    assert off(got, want) < 1e-5 and np.abs(got - want).max() < 1e-4
    if epi != _lib.EPI_NONE:
        assert (np.abs(z) > limit).mean() > 0.2


# ------------------------------------------------------------------ matrix memory
class Memory:
    """Device operands of one layer's recurrence for `batch` sequences, and the oracle's on the host."""

    def __init__(self, heads, d, e, batch, seed, cap=8.0, eps=1e-5, forget=(-2.0, 6.0), inp=(-4.0, 4.0)):
        rng = np.random.default_rng(seed)
        self.m, self.B, self.cap, self.eps, self.rng = (heads, d, e), batch, cap, eps, rng
        self.nb = 2 * heads * (d + e)
        self.ld = (self.nb + 2 * heads + 3) // 4 * 4
        self.ib, self.fb = (rng.uniform(*r, heads).astype(np.float32) for r in (inp, forget))
        self.norm = rng.uniform(0.5, 1.5, heads * e).astype(np.float32)
        self.keep = [dev(a) for a in (self.ib, self.fb, self.norm)]
        self.w = _lib.CMemoryWeights(*[k.ptr for k in self.keep], eps)
        self.s = _lib.CMemoryShape(heads, d, e, self.ld, cap)
        self.state = [DeviceArray(x).zero_() for x in ((batch, heads, d, e), (batch, heads, d), (batch, heads))]

    def inputs(self, n):
        p = self.rng.normal(size=(self.B, n, self.ld)).astype(np.float32)
        p[..., self.nb:] *= 3.0
        p[..., self.nb + 2 * self.m[0]:] = np.nan  # padding columns are never used
        return p

    def prompt(self, p, chunked):
        H, d, e = self.m
        out, x = DeviceArray((self.B, p.shape[1], H * e)), dev(np.ascontiguousarray(p))
        _check(_lib.load().coeus_op_memory_prompt(C.byref(self.s), C.byref(self.w), x.ptr, *[a.ptr for a in self.state], self.B,
                                                  p.shape[1], chunked, out.ptr, None))
        return out.to_host()

    def step(self, p):
        H, d, e = self.m
        out, x = DeviceArray((self.B, H * e)), dev(np.ascontiguousarray(p))
        _check(_lib.load().coeus_op_memory_step(C.byref(self.s), C.byref(self.w), x.ptr, *[a.ptr for a in self.state], self.B,
                                                out.ptr, None))
        return out.to_host()

    def want(self, p):
        """Outputs, and final states as (S, n) times e^m and m, of whole sequences p [B, T, ld]."""
        H, d, e = self.m
        outs, states = [], []
        p = p.astype(np.float64)
        for b in range(self.B):
            x = p[b]
            q, k = (x[:, i * H * d:(i + 1) * H * d].reshape(-1, H, d) for i in (0, 1))
            v, g = (x[:, 2 * H * d + i * H * e:2 * H * d + (i + 1) * H * e].reshape(-1, H, e) for i in (0, 1))
            li = L.soft_cap(x[:, self.nb:self.nb + H] + self.ib.astype(np.float64), self.cap)
            lf = L.log_sigmoid(L.soft_cap(x[:, self.nb + H:self.nb + 2 * H] + self.fb.astype(np.float64), self.cap))
            o, st = np.zeros_like(v), []
            for h in range(H):
                o[:, h], s = L.matrix_memory(q[:, h] * d ** -0.5, k[:, h], v[:, h], li[:, h], lf[:, h])
                st.append(s)
            o = L.rms_norm(o, self.norm.astype(np.float64).reshape(H, e), self.eps) * L.sigmoid(g)
            outs.append(o.reshape(-1, H * e))
            states.append([np.stack([s[j] for s in st]) for j in range(3)])
        return np.stack(outs), [np.stack([s[j] for s in states]) for j in range(3)]

    def state_off(self, want):
        return max(off(a.to_host(), w) for a, w in zip(self.state, want))


MEMORY = [(4, 24, 64), (3, 20, 24), (2, 128, 128), (3, 80, 96), (1, 200, 40), (1, 256, 256), (5, 16, 33), (1, 8, 8), (2, 300, 20), (1, 12, 600),
          (2, 9, 5), (1, 4, 1024), (2, 36, 132), (1, 512, 16), (2, 48, 4)]


@pytest.mark.parametrize("shape", MEMORY)
@pytest.mark.parametrize("n", [1, 47, 64, 65, 150])
@pytest.mark.parametrize("chunked", [0, 1])
def test_memory_prompt(shape, n, chunked):
    t = Memory(*shape, batch=2, seed=n, cap=30.0 if n == 65 else 8.0)
    p = t.inputs(n)
    got, (want, S) = t.prompt(p, chunked), t.want(p)
    assert off(got, want) < 2e-5 and t.state_off(S) < 2e-5


@pytest.mark.parametrize("shape", MEMORY)
def test_memory_steps(shape):
    t = Memory(*shape, batch=2, seed=3)
    p = t.inputs(12)
    want, S = t.want(p)
    got = np.stack([t.step(p[:, i]) for i in range(12)], axis=1)
    assert max(off(got[:, i], want[:, i]) for i in range(12)) < 2e-5 and t.state_off(S) < 2e-5


@pytest.mark.parametrize("shape", MEMORY[:7])
def test_memory_portions_and_steps(shape):
    """A sequence cut into portions from one token to several chunks, single steps in between."""
    t = Memory(*shape, batch=3, seed=7)
    cuts = [2, 1, 3, 64, 2, 70, 1, 1, 5, 130, 2]
    p = t.inputs(sum(cuts))
    want, S = t.want(p)
    pos, got = 0, []
    for c in cuts:
        x = p[:, pos:pos + c]
        got.append(t.step(x[:, 0])[:, None] if c == 1 else t.prompt(x, 1))
        pos += c
    got = np.concatenate(got, axis=1)
    assert max(off(got[:, i], want[:, i]) for i in range(pos)) < 1e-4 and t.state_off(S) < 2e-5


@pytest.mark.parametrize("n", [4096 + 130, 4096 + 1])
def test_memory_long_prompt(n):
    """More tokens than chunk states are held for at once."""
    t = Memory(2, 8, 12, batch=1, seed=n)
    p = t.inputs(n)
    want, S = t.want(p)
    got = t.prompt(p, 1)
    assert off(got, want) < 2e-5 and off(got[:, 4000:], want[:, 4000:]) < 2e-5 and t.state_off(S) < 2e-5


def test_memory_long_decoding():
    t = Memory(4, 32, 48, batch=2, seed=11)
    p = t.inputs(400)
    want, S = t.want(p)
    got = np.stack([t.step(p[:, i]) for i in range(400)], axis=1)
    assert off(got, want) < 2e-5 and off(got[:, -20:], want[:, -20:]) < 5e-5 and t.state_off(S) < 2e-5


@pytest.mark.parametrize("way", ["chunked", "scan", "steps"])
def test_memory_recalls_a_far_write(way):
    """One token writes strongly into a memory that forgets nothing; hundreds of tokens and several chunks later
    its key reads it back.  A lost, decayed or wrongly scaled state would show."""
    t = Memory(2, 16, 24, batch=1, seed=5, cap=40.0)
    H, d, e = t.m
    n = 300
    p = t.inputs(n)
    p[..., t.nb:t.nb + H] = -1e4                    # nobody writes ..
    p[:, 3, t.nb:t.nb + H] = 8.0                    # .. except token 3
    p[..., t.nb + H:t.nb + 2 * H] = 1e4             # nobody forgets
    p[:, n - 1, :H * d] = p[:, 3, H * d:2 * H * d]  # the last query is its key
    want, S = t.want(p)
    got = t.prompt(p, way == "chunked") if way != "steps" else np.stack([t.step(p[:, i]) for i in range(n)], axis=1)
    v = p[0, 3, 2 * H * d:2 * H * d + H * e].reshape(H, e)
    read = (got[0, -1] / t.norm / L.sigmoid(p[0, -1, 2 * H * d + H * e:t.nb])).reshape(H, e)
    assert off(got[:, -1], want[:, -1]) < 1e-4 and t.state_off(S) < 1e-5
    for h in range(H):
        assert np.corrcoef(read[h], v[h])[0, 1] > 0.9999


@pytest.mark.parametrize("way", ["chunked", "scan", "steps"])
def test_memory_maximum_starts_at_zero(way):
    """Weak input gates: the running maximum, which starts at 0 and falls with the forget gates, and not the gate
    itself scales the first tokens' state; the normaliser's floor e^-m is what divides."""
    t = Memory(3, 8, 12, batch=2, seed=9, inp=(-7.0, -5.0), forget=(3.0, 5.0), eps=1e-12)
    p = t.inputs(60)
    want, S = t.want(p)
    got = t.prompt(p, way == "chunked") if way != "steps" else np.stack([t.step(p[:, i]) for i in range(60)], axis=1)
    assert max(off(got[:, i], want[:, i]) for i in range(60)) < 5e-5 and t.state_off(S) < 2e-5
    raw, st = Memory.want(t, p[:, :1])
    assert (st[2] < 0).all() and (st[2] > -1).all()  # the maximum behind the first token is the forget gate's


def test_memory_sequences_do_not_meet():
    t = Memory(2, 24, 16, batch=3, seed=2)
    p = t.inputs(100)
    every = t.prompt(p, 1)
    for b in range(3):
        one = Memory(2, 24, 16, batch=1, seed=2)
        assert np.array_equal(one.prompt(p[b:b + 1], 1)[0], every[b])


def test_memory_refuses_bad_shapes():
    t = Memory(2, 8, 8, batch=1, seed=1)
    x, out, lib = dev(t.inputs(2)), DeviceArray((2, 16)), _lib.load()
    for field, value in (("heads", 0), ("dim", 0), ("dim", 513), ("vdim", 1025), ("in_ld", 8), ("gate_cap", 0.0)):
        s = _lib.CMemoryShape(*[getattr(t.s, f) for f, _ in _lib.CMemoryShape._fields_])
        setattr(s, field, value)
        st = [a.ptr for a in t.state]
        assert lib.coeus_op_memory_step(C.byref(s), C.byref(t.w), x.ptr, *st, 1, out.ptr, None) == _lib.INVALID_INPUT
        assert lib.coeus_op_memory_prompt(C.byref(s), C.byref(t.w), x.ptr, *st, 1, 2, 1, out.ptr, None) == _lib.INVALID_INPUT


# ------------------------------------------------------------------ attention whose values are its keys
class SharedKv:
    """Sequences through the operators with a ring on the device; the projections so far on the host."""

    def __init__(self, H, G, d, window, cap, batch, bf16, seed, scale=None, slope_range=8.0, sharp=2.0):
        rng = np.random.default_rng(seed)
        self.m, self.cap, self.B, self.bf16, self.rng = (H, G, d, window), cap, batch, bf16, rng
        self.scale, self.range, self.eps = scale or d ** -0.5, slope_range, 1e-4
        self.used = (2 * H + G) * d
        self.ld = (self.used + 3) // 4 * 4
        self.wq, self.wk = (rng.uniform(0.5, 1.5, n) * sharp for n in (H * d, G * d))
        wqk = self.wq.reshape(H, d) * self.wk.reshape(G, d)[np.arange(H) // (H // G)]
        self.d_w = dev(wqk.reshape(-1), np.float32)
        row = _lib.load().coeus_shared_kv_row_len(G, d)
        self.ring = DeviceArray((batch, cap, row), np.uint16 if bf16 else np.float32).zero_()
        self.s = _lib.CSharedKvShape(H, G, d, window or 0, self.ld, self.scale, slope_range)
        self.seen = np.zeros((batch, 0, self.used))

    def inputs(self, n, standout=(), boost=6.0):
        """standout (row, key): positions behind those fed so far; the query of `row` asks for `key`'s key."""
        H, G, d, _ = self.m
        p = self.rng.normal(size=(self.B, n, self.ld)).astype(np.float32)
        p[..., self.used:] = np.nan
        for row, key in standout:
            k = p[:, key, H * d:(H + G) * d].reshape(self.B, G, d)
            p[:, row, :H * d] = boost * k[:, np.arange(H) // (H // G)].reshape(self.B, -1)
        if self.bf16:  # (keys between two bf16 numbers would hide what is tested)
            p[..., H * d:(H + G) * d] = bf16_round(p[..., H * d:(H + G) * d])
        return p

    def feed(self, p, decode=False):
        H, G, d, _ = self.m
        n, pos = p.shape[1], self.seen.shape[1]
        out, x, lib, dt = DeviceArray((self.B, n, H * d)), dev(np.ascontiguousarray(p)), _lib.load(), _lib.KV_BF16 if self.bf16 else _lib.KV_F32
        if decode:
            _check(lib.coeus_op_shared_kv_decode(C.byref(self.s), dt, x.ptr, self.d_w.ptr, self.eps, self.ring.ptr, self.cap, self.B, pos,
                                                 out.ptr, None))
        else:
            _check(lib.coeus_op_shared_kv_prompt(C.byref(self.s), dt, x.ptr, self.d_w.ptr, self.eps, self.ring.ptr, self.cap, self.B, n, pos,
                                                 out.ptr, None))
        self.seen = np.concatenate([self.seen, p[..., :self.used].astype(np.float64)], axis=1)
        return out.to_host()

    def want(self, window=0):
        H, G, d, own = self.m
        window, T, outs = own if window == 0 else window, self.seen.shape[1], []
        slopes = L.distance_slopes(H) if self.range else np.zeros(H)
        for x in self.seen:
            v = x[:, H * d:(H + G) * d]
            q = L.rms_norm(x[:, :H * d], self.wq, self.eps).reshape(T, H, d)
            k, v = L.rms_norm(v, self.wk, self.eps).reshape(T, G, d), v.reshape(T, G, d)
            o = np.stack([L.biased_attention(q[:, h], k[:, h // (H // G)], v[:, h // (H // G)], self.scale, window, slopes[h])
                          for h in range(H)], axis=1).reshape(T, H * d)
            outs.append(o * L.sigmoid(x[:, (H + G) * d:]))
        return np.stack(outs)


# f32 is exact; bf16 prompts round the weighted queries, and a score of 10 then moves by a hundredth
KV_LIMIT = {False: 1e-5, True: 1.5e-2}
KV_SHAPES = [(6, 3, 24), (4, 4, 64), (8, 1, 48), (3, 1, 9), (2, 2, 128), (4, 2, 200), (5, 1, 256), (16, 2, 40), (2, 1, 12), (7, 7, 8)]


@pytest.mark.parametrize("bf16", [False, True])
@pytest.mark.parametrize("shape", KV_SHAPES)
@pytest.mark.parametrize("window,cuts", [(None, [70]), (1, [9, 2]), (2, [33, 5]), (32, [31, 130]), (33, [70, 40]), (48, [47, 2, 3]), (90, [150, 110]),
                                         (200, [40, 60])])
def test_shared_kv_prompt(shape, window, cuts, bf16):
    cap = min(window or 10 ** 9, sum(cuts))
    t = SharedKv(*shape, window, cap, 2, bf16, seed=sum(cuts))
    got = np.concatenate([t.feed(t.inputs(c)) for c in cuts], axis=1)
    assert off(got, t.want()) < KV_LIMIT[bf16]


@pytest.mark.parametrize("bf16", [False, True])
@pytest.mark.parametrize("shape", KV_SHAPES)
@pytest.mark.parametrize("window,cap,batch", [(5, 5, 1), (64, 64, 2), (65, 65, 1), (1, 1, 3), (None, 100, 2), (200, 80, 1)])
def test_shared_kv_decode(shape, window, cap, batch, bf16):
    """From the first token past the point where the ring comes round (or to the ring's end)."""
    t = SharedKv(*shape, window, cap, batch, bf16, seed=cap)
    steps = cap if window is None or cap < window else 2 * cap + 3
    got = np.concatenate([t.feed(t.inputs(1), decode=True) for _ in range(steps)], axis=1)
    want = t.want()
    assert max(off(got[:, i], want[:, i]) for i in range(steps)) < (1e-5 if not bf16 else 1e-4)


@pytest.mark.parametrize("bf16", [False, True])
def test_shared_kv_mixed_portions(bf16):
    t = SharedKv(6, 2, 32, 37, 37, 2, bf16, seed=1)
    cuts = [2, 1, 1, 40, 2, 3, 1, 36, 37, 38, 1, 1, 2, 100, 1]
    got = np.concatenate([t.feed(t.inputs(c), decode=c == 1) for c in cuts], axis=1)
    want = t.want()
    assert max(off(got[:, i], want[:, i]) for i in range(sum(cuts))) < 5 * KV_LIMIT[bf16]


@pytest.mark.parametrize("bf16", [False, True])
@pytest.mark.parametrize("batch,cap,shape", [(1, 1000, (4, 2, 64)), (2, 3000, (16, 2, 32)), (1, 500, (6, 6, 136)), (1, 700, (3, 1, 20))])
def test_shared_kv_decode_many_shares(batch, cap, shape, bf16):
    """Rings that many workgroups share, behind a prompt, before and after they come round."""
    t = SharedKv(*shape, cap, cap, batch, bf16, seed=cap, slope_range=0.0)
    t.feed(t.inputs(cap - 4))
    got = np.concatenate([t.feed(t.inputs(1), decode=True) for _ in range(9)], axis=1)
    assert off(got, t.want()[:, -9:]) < (1e-5 if not bf16 else 1e-4)


@pytest.mark.parametrize("bf16", [False, True])
@pytest.mark.parametrize("window", [31, 32, 33, 64])
def test_shared_kv_edges_in_prompts(window, bf16):
    """One outstanding key just inside and just outside a row's window, the row's own key, and the very first
    key, at rows whose window starts at, before and behind a tile's edge."""
    n = 140
    for row in (window - 1, window, 96, 127, 128, n - 1):
        for key in (row, max(0, row - window + 1), row - window, 0):
            if key < 0:
                continue
            t = SharedKv(2, 1, 32, window, window, 1, bf16, seed=row, slope_range=0.0)
            got = t.feed(t.inputs(n, [(row, key)]))
            want = t.want()
            assert off(got[:, row], want[:, row]) < 2 * KV_LIMIT[bf16], (row, key)
            if row - window < key < row:  # the case shows: one position less and the row returns something else
                assert key > row - window + 1 or off(t.want(window - 1)[:, row], want[:, row]) > 0.5
            if key == row - window:
                assert off(t.want(window + 1)[:, row], want[:, row]) > 0.5


@pytest.mark.parametrize("bf16", [False, True])
def test_shared_kv_edge_in_decoding(bf16):
    """A key that every later query of this test asks for: seen window - 1 steps later and not one step on."""
    W = 37
    t = SharedKv(4, 2, 32, W, W, 1, bf16, seed=3, slope_range=0.0)
    n = 5 + W + 3
    p = t.inputs(n, [(r, 4) for r in range(5, n)])
    got = np.concatenate([t.feed(p[:, :5])] + [t.feed(p[:, i:i + 1], decode=True) for i in range(5, n)], axis=1)
    want, wide = t.want(), t.want(W + 1)
    assert max(off(got[:, i], want[:, i]) for i in range(5, n)) < (1e-5 if not bf16 else 1e-3)
    assert off(wide[:, 4 + W], want[:, 4 + W]) > 0.5 and off(wide[:, 3 + W], want[:, 3 + W]) < 1e-6


@pytest.mark.parametrize("bf16", [False, True])
@pytest.mark.parametrize("decode", [False, True])
def test_shared_kv_far_key_among_hundreds(decode, bf16):
    """Distance costs slope times it, exactly: a key 600 positions back that outweighs all others in the heads with
    small slopes, and by what remains in the others; a slope that is off by a hundredth shows."""
    t = SharedKv(4, 2, 32, None, 640, 1, bf16, seed=8, scale=0.3)
    p = t.inputs(640, [(r, 20) for r in (620, 621, 622)])
    got = t.feed(p[:, :600])
    got = np.concatenate([t.feed(p[:, i:i + 1], decode=True) for i in range(600, 640)] if decode else [t.feed(p[:, 600:])], axis=1)
    want = t.want()
    assert max(off(got[:, i - 600], want[:, i]) for i in (620, 621, 622)) < (2e-5 if not bf16 else 4e-2)
    v = t.seen[0, 20, 4 * 32:6 * 32].reshape(2, 32)
    last = (want[0, 620] / L.sigmoid(t.seen[0, 620, 6 * 32:])).reshape(4, 32)[3]
    assert off(last, v[1]) < 0.2  # (it does outweigh them)


def test_shared_kv_refusals():
    lib, t = _lib.load(), SharedKv(4, 2, 16, 8, 8, 1, False, seed=1)
    x, out = dev(t.inputs(2)), DeviceArray((1, 2, 64))

    def both(s, cap=8, pos=0):
        a = C.byref(s), _lib.KV_F32, x.ptr, t.d_w.ptr, 1e-5, t.ring.ptr, cap, 1
        assert lib.coeus_op_shared_kv_prompt(*a, 2, pos, out.ptr, None) == _lib.INVALID_INPUT
        assert lib.coeus_op_shared_kv_decode(*a, pos, out.ptr, None) == _lib.INVALID_INPUT
    for field, value in (("kv_heads", 0), ("kv_heads", 3), ("dim", 257), ("in_ld", 100), ("heads", 0)):
        s = _lib.CSharedKvShape(*[getattr(t.s, f) for f, _ in _lib.CSharedKvShape._fields_])
        setattr(s, field, value)
        both(s)
    both(t.s, cap=9)
    both(t.s, cap=4, pos=5)
    assert lib.coeus_op_shared_kv_decode(C.byref(t.s), _lib.KV_F16, x.ptr, t.d_w.ptr, 1e-5, t.ring.ptr, 8, 1, 0, out.ptr,
                                         None) == _lib.INVALID_INPUT
    assert lib.coeus_shared_kv_row_len(3, 16) == 56 and lib.coeus_shared_kv_row_len(1, 9) == 24
