"""GPU checks of the layered models: each mechanism alone through the operator entry points, then whole
models through folders, sessions and generation, against the plain restatement in oracle/layered.py."""
import ctypes as C
import json

import numpy as np
import pytest

from coeus_amd import BasicGenerationConfig, LayeredConfig, PLUGINS, ProcessingError, _lib, load_model, trace
from coeus_amd.device import DeviceArray
from coeus_amd.plugin import _check
from gpu_util import dev
from layered_util import (BOFIRAX, CONFIGS, ZEKILIX, bf16_round, config, delta, hyper_config, latent, memory, shared_kv, weights,
                          write_folder)
from oracle import layered as L

pytestmark = pytest.mark.gpu


def off(got, want):
    """Root mean square of the difference over the root mean square of the expected values."""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    return float(np.sqrt(np.mean((got - want) ** 2)) / max(np.sqrt(np.mean(want ** 2)), 1e-30))


def bf16_dev(a):
    return dev((np.ascontiguousarray(bf16_round(a)).view(np.uint32) >> 16).astype(np.uint16))


# ------------------------------------------------------------------ norm behind a sublayer
@pytest.mark.parametrize("rows,hidden,with_ls", [(1, 64, True), (5, 130, True), (3, 4096, False), (2, 8196, True), (700, 96, True)])
def test_norm_residual(rows, hidden, with_ls):
    rng = np.random.default_rng(rows + hidden)
    y, h = rng.normal(size=(rows, hidden)) * 3, rng.normal(size=(rows, hidden))
    s, ls = rng.uniform(0.5, 1.5, hidden), rng.uniform(0.5, 1.5, hidden)
    dy, dh, ds, dl = (dev(a, np.float32) for a in (y, h, s, ls))
    _check(_lib.load().coeus_op_norm_residual(dy.ptr, rows, hidden, ds.ptr, dl.ptr if with_ls else None, 1e-3, dh.ptr, None))
    assert off(dh.to_host(), h + L.rms_norm(y, s, 1e-3) * (ls if with_ls else 1.0)) < 1e-6


# ------------------------------------------------------------------ gated delta rule
class Delta:
    """Device operands of one layer's recurrence for `batch` sequences, and the oracle's on the host."""

    def __init__(self, heads, kv_heads, d, e, taps, batch, seed, fast=False, eps=1e-5):
        rng = np.random.default_rng(seed)
        self.m, self.B, self.eps, self.rng = (heads, kv_heads, d, e, taps), batch, eps, rng
        self.C = 2 * kv_heads * d + heads * e
        self.ld = (self.C + heads * e + 2 * heads + 3) // 4 * 4
        self.conv = rng.normal(0, 0.6, (self.C, taps)).astype(np.float32)
        self.a_log = rng.uniform(-4, 3.0 if fast else 0.5, heads).astype(np.float32)
        self.dt = rng.uniform(-3, 2.0 if fast else 0.0, heads).astype(np.float32)
        self.norm = rng.uniform(0.5, 1.5, e).astype(np.float32)
        self.keep = [dev(np.ascontiguousarray(self.conv.T)), dev(np.exp(self.a_log)), dev(self.dt), dev(self.norm)]
        self.w = _lib.CDeltaWeights(*[k.ptr for k in self.keep], eps)
        self.s = _lib.CDeltaShape(heads, kv_heads, d, e, taps, self.ld)
        self.state, self.ring = DeviceArray((batch, heads, d, e)).zero_(), DeviceArray((batch, taps, self.C)).zero_()

    def inputs(self, n):
        p = self.rng.normal(size=(self.B, n, self.ld)).astype(np.float32)
        p[..., self.C + self.m[0] * self.m[3] + 2 * self.m[0]:] = np.nan  # padding columns are never used
        return p

    def prompt(self, p, pos0, chunked):
        out, x = DeviceArray((self.B, p.shape[1], self.m[0] * self.m[3])), dev(p)
        _check(_lib.load().coeus_op_delta_prompt(C.byref(self.s), C.byref(self.w), x.ptr, self.state.ptr, self.ring.ptr, self.B,
                                                 p.shape[1], pos0, chunked, out.ptr, None))
        return out.to_host()

    def step(self, p, pos):
        out, x = DeviceArray((self.B, self.m[0] * self.m[3])), dev(p)
        _check(_lib.load().coeus_op_delta_step(C.byref(self.s), C.byref(self.w), x.ptr, self.state.ptr, self.ring.ptr, self.B, pos,
                                               out.ptr, None))
        return out.to_host()

    def want(self, p):
        """Outputs and final states of whole sequences p [B, T, ld], one head at a time."""
        H, KH, d, e, _ = self.m
        outs, states, p = [], [], p.astype(np.float64)
        conv, nb = self.conv.astype(np.float64), self.C + H * e
        for b in range(self.B):
            x = p[b]
            y = L.short_conv(x[:, :self.C], conv)
            q = L.unit(y[:, :KH * d].reshape(-1, KH, d)) * d ** -0.5
            k = L.unit(y[:, KH * d:2 * KH * d].reshape(-1, KH, d))
            v = y[:, 2 * KH * d:].reshape(-1, H, e)
            beta = L.sigmoid(x[:, nb:nb + H])
            decay = np.exp(-np.exp(self.a_log.astype(np.float64)) * L.softplus(x[:, nb + H:nb + 2 * H] + self.dt.astype(np.float64)))
            o, S = np.zeros_like(v), np.zeros((H, d, e))
            for h in range(H):
                o[:, h], S[h] = L.delta_rule(q[:, h // (H // KH)], k[:, h // (H // KH)], v[:, h], beta[:, h], decay[:, h])
            o = L.rms_norm(o, self.norm.astype(np.float64), self.eps) * L.silu(x[:, self.C:nb]).reshape(-1, H, e)
            outs.append(o.reshape(-1, H * e))
            states.append(S)
        return np.stack(outs), np.stack(states)


SHAPES = [(4, 2, 24, 64, 4), (6, 3, 20, 24, 3), (2, 2, 128, 128, 4), (3, 1, 80, 96, 2), (2, 1, 200, 40, 1), (5, 5, 16, 33, 5),
          (1, 1, 8, 8, 4), (2, 2, 256, 16, 2)]


@pytest.mark.parametrize("shape", SHAPES)
@pytest.mark.parametrize("n", [1, 47, 64, 65, 150])
@pytest.mark.parametrize("chunked", [0, 1])
def test_delta_prompt(shape, n, chunked):
    t = Delta(*shape, batch=2, seed=n, fast=n == 65)
    p = t.inputs(n)
    got, (want, S) = t.prompt(p, 0, chunked), t.want(p)
    assert off(got, want) < 2e-5 and off(t.state.to_host(), S) < 2e-5


@pytest.mark.parametrize("shape", SHAPES[:6])
def test_delta_portions_and_steps(shape):
    """A sequence cut into portions from one token to several chunks, single steps in between: outputs of
    every token, and the state at the end."""
    t = Delta(*shape, batch=3, seed=7)
    cuts = [2, 1, 3, 64, 2, 70, 1, 1, 5, 130, 2]
    p = t.inputs(sum(cuts))
    want, S = t.want(p)
    pos, got = 0, []
    for i, c in enumerate(cuts):
        x = np.ascontiguousarray(p[:, pos:pos + c])
        got.append(t.step(x[:, 0], pos)[:, None] if c == 1 else t.prompt(x, pos, 1))
        pos += c
    got = np.concatenate(got, axis=1)
    assert max(off(got[:, i], want[:, i]) for i in range(pos)) < 5e-5 and off(t.state.to_host(), S) < 2e-5


def test_delta_long_decoding():
    t = Delta(4, 2, 32, 48, 4, batch=2, seed=11)
    p = t.inputs(400)
    want, S = t.want(p)
    got = np.stack([t.step(np.ascontiguousarray(p[:, i]), i) for i in range(400)], axis=1)
    assert off(got, want) < 2e-5 and off(got[:, -20:], want[:, -20:]) < 5e-5 and off(t.state.to_host(), S) < 2e-5


def test_delta_recalls_a_far_write():
    """One key written at full strength into a state that does not decay is read back hundreds of tokens
    (and several chunks) later: what a lost or decayed state would hide."""
    t = Delta(1, 1, 16, 16, 1, batch=1, seed=5)
    H, KH, d, e, _ = t.m
    t.a_log[:] = -20.0
    t.keep[1] = dev(np.exp(t.a_log))
    t.w.exp_a_dev = t.keep[1].ptr
    n = 300
    p = t.inputs(n)
    nb = t.C + H * e
    p[..., nb] = -30.0                       # nobody writes ..
    p[0, 3, nb] = 30.0                       # .. except token 3
    p[0, n - 1, :d] = p[0, 3, d:2 * d] * t.conv[d:2 * d, 0] / t.conv[:d, 0]  # the last query is its key
    want, S = t.want(p)
    got = t.prompt(p, 0, 1)
    assert off(got[0, -1], want[0, -1]) < 1e-4 and off(t.state.to_host(), S) < 1e-5
    assert np.abs(S).max() > 0.05 and np.abs(want[0, -1]).max() > 0.01


def test_delta_refuses_bad_shapes():
    t = Delta(2, 2, 8, 8, 2, batch=1, seed=1)
    for field, value in (("kv_heads", 0), ("kv_heads", 3), ("dim", 257), ("conv", 17), ("in_ld", 8)):
        s = _lib.CDeltaShape(*[getattr(t.s, f) for f, _ in _lib.CDeltaShape._fields_])
        setattr(s, field, value)
        x, out = dev(t.inputs(1)), DeviceArray((1, 16))
        for rc in (_lib.load().coeus_op_delta_step(C.byref(s), C.byref(t.w), x.ptr, t.state.ptr, t.ring.ptr, 1, 0, out.ptr, None),
                   _lib.load().coeus_op_delta_prompt(C.byref(s), C.byref(t.w), x.ptr, t.state.ptr, t.ring.ptr, 1, 1, 0, 1, out.ptr, None)):
            assert rc == _lib.INVALID_INPUT


# ------------------------------------------------------------------ windowed attention
def window_case(heads, d, e, window, n, hist, batch, bf16, seed, standout=None, scale=None):
    """standout (row, key): that score is far above all others."""
    rng = np.random.default_rng(seed)
    T = hist + n
    q, k = rng.normal(size=(batch, n, heads, d)), rng.normal(size=(batch, T, heads, d))
    v = rng.normal(size=(batch, T, heads, e))
    for row, key in standout or ():
        u = rng.normal(size=(heads, d))
        u /= np.linalg.norm(u, axis=-1, keepdims=True)
        q[:, row] = 12 * u
        k[:, key] = 12 * u
    r = bf16_round if bf16 else (lambda a: np.asarray(a, np.float32))
    q, k, v = r(q), r(k), r(v)
    kv = np.concatenate([k.reshape(batch * T, -1), v.reshape(batch * T, -1)], axis=1)
    put = bf16_dev if bf16 else (lambda a: dev(a, np.float32))
    dq, dkv, out = put(q.reshape(batch * n, -1)), put(kv), DeviceArray((batch, n, heads, e))
    s = _lib.CLatentShape(heads, d, e, 1, 1, window or 0, scale or d ** -0.5)
    _check(_lib.load().coeus_op_window_attention(C.byref(s), _lib.KV_BF16 if bf16 else _lib.KV_F32, dq.ptr, dkv.ptr, batch, n, hist,
                                                 out.ptr, None))
    want = np.zeros((batch, n, heads, e))
    for b in range(batch):
        for h in range(heads):
            full = np.zeros((T, d))
            full[hist:] = q[b, :, h]
            want[b, :, h] = L.masked_attention(full, k[b, :, h].astype(np.float64), v[b, :, h].astype(np.float64),
                                               scale or d ** -0.5, window)[hist:]
    return out.to_host(), want


@pytest.mark.parametrize("bf16", [False, True])
@pytest.mark.parametrize("heads,d,e", [(3, 64, 72), (2, 24, 16), (2, 128, 128), (2, 20, 12), (1, 96, 256), (2, 256, 64), (8, 40, 136)])
@pytest.mark.parametrize("window,n,hist", [(None, 70, 0), (1, 9, 0), (2, 33, 1), (32, 130, 31), (33, 40, 32), (48, 2, 47), (90, 260, 89)])
def test_window_attention(heads, d, e, window, n, hist, bf16):
    got, want = window_case(heads, d, e, window, n, hist, 2, bf16, seed=n)
    assert off(got, want) < (2e-6 if not bf16 else 2e-5)  # bf16 inputs are exact; weights and sums are f32


@pytest.mark.parametrize("bf16", [False, True])
@pytest.mark.parametrize("window", [31, 32, 33, 64])
def test_window_attention_edges(window, bf16):
    """One outstanding key just inside and just outside a row's window, the row's own key, and the very first
    key, at rows whose window starts at, before and behind a tile's edge; negative scales turn them round."""
    n = 140
    for row in (window - 1, window, 96, 127, 128, n - 1):
        for key in (row, max(0, row - window + 1), row - window, 0):
            if key < 0:
                continue
            got, want = window_case(2, 32, 48, window, n, 0, 1, bf16, seed=row, standout=[(row, key)])
            assert off(got[0, row], want[0, row]) < 1e-4, (row, key)
            seen = row - window < key <= row
            own = window_case(2, 32, 48, window, n, 0, 1, bf16, seed=row)[1]
            if seen:  # the case shows: that key's weight is what the row returns
                assert off(want[0, row], own[0, row]) > 0.1
    got, want = window_case(2, 32, 48, window, n, 0, 1, bf16, seed=1, scale=-0.3)
    assert off(got, want) < 1e-4


# ------------------------------------------------------------------ latent attention of a decode step
class LatentDecode:
    def __init__(self, heads, d, e, qr, R, window, cap, batch, bf16, seed):
        rng = np.random.default_rng(seed)
        self.m, self.B, self.cap, self.bf16, self.rng = (heads, d, e, qr, R, window), batch, cap, bf16, rng
        self.r = bf16_round if bf16 else (lambda a: np.asarray(a, np.float32))
        self.ld = (qr + R + 3) // 4 * 4
        self.ukv = self.r(rng.normal(size=(heads * (d + e), R)) / np.sqrt(R))
        self.scale = rng.uniform(0.5, 1.5, R).astype(np.float32)
        put = bf16_dev if bf16 else (lambda a: dev(a, np.float32))
        self.d_ukv, self.d_scale = put(self.ukv), dev(self.scale)
        self.cache = DeviceArray((batch, cap, R), np.uint16 if bf16 else np.float32).zero_()
        self.lat = []  # the latents so far, [batch, R] each
        self.s = _lib.CLatentShape(heads, d, e, qr, R, window or 0, d ** -0.5)

    def step(self, pos, q=None, boost=1.0):
        H, d, e, qr, R, window = self.m
        q = self.rng.normal(size=(self.B, H, d)) * 3 if q is None else q
        q = q.astype(np.float32)
        proj = self.rng.normal(size=(self.B, self.ld)).astype(np.float32) * boost
        c = self.r(L.rms_norm(proj[:, qr:qr + R].astype(np.float64), self.scale.astype(np.float64), 1e-5))
        self.lat.append(c.astype(np.float64))
        dq, dp, out = dev(q), dev(proj), DeviceArray((self.B, H, e))
        _check(_lib.load().coeus_op_latent_decode(C.byref(self.s), _lib.KV_BF16 if self.bf16 else _lib.KV_F32, dq.ptr, dp.ptr,
                                                  self.d_scale.ptr, 1e-5, self.d_ukv.ptr, self.cache.ptr, self.cap, self.B, pos,
                                                  out.ptr, None))
        lo = 0 if window is None else max(0, pos - window + 1)
        c = np.stack(self.lat[lo:], axis=1)  # [B, keys, R]
        uk, uv = self.ukv[:H * d].reshape(H, d, R).astype(np.float64), self.ukv[H * d:].reshape(H, e, R).astype(np.float64)
        want = np.zeros((self.B, H, e))
        for b in range(self.B):
            for h in range(H):
                s = (c[b] @ uk[h].T) @ q[b, h].astype(np.float64) * d ** -0.5
                a = np.exp(s - s.max())
                want[b, h] = (a / a.sum()) @ (c[b] @ uv[h].T)
        return out.to_host(), want


@pytest.mark.parametrize("bf16", [False, True])
@pytest.mark.parametrize("heads,d,e,qr,R,window,cap,batch", [
    (3, 24, 40, 20, 32, 5, 5, 1), (4, 64, 72, 48, 96, 64, 64, 2), (2, 32, 16, 8, 512, 65, 65, 1), (17, 16, 24, 12, 64, 70, 70, 3),
    (2, 40, 48, 12, 1024, 9, 9, 1), (2, 18, 10, 7, 40, 6, 6, 2), (3, 32, 32, 16, 64, None, 90, 2), (2, 8, 8, 4, 160, 200, 80, 16),
    (2, 16, 264 - 64, 8, 544, 3, 3, 1)])
def test_latent_decode(heads, d, e, qr, R, window, cap, batch, bf16):
    """From the first token past the point where the ring comes round (or to its end, where the context is
    shorter than the window)."""
    t = LatentDecode(heads, d, e, qr, R, window, cap, batch, bf16, seed=R)
    steps = cap if window is None or cap < window else 2 * cap + 3
    for pos in range(steps):
        got, want = t.step(pos)
        # (a latent that lands between two bf16 numbers may be rounded to the other one)
        assert off(got, want) < (5e-6 if not bf16 else 2e-3), pos


@pytest.mark.parametrize("bf16", [False, True])
def test_latent_decode_window_edge(bf16):
    """A latent that every query of this test asks for is seen window - 1 steps later and not one step on."""
    H, d, e, R, W = 2, 16, 24, 64, 37
    t = LatentDecode(H, d, e, 8, R, W, W, 1, bf16, seed=3)
    for pos in range(5):
        t.step(pos)
    uk = t.ukv[:H * d].reshape(H, d, R).astype(np.float64)
    q = np.stack([[40 * uk[h] @ t.lat[4][0] / np.linalg.norm(uk[h] @ t.lat[4][0]) for h in range(H)]])
    before = None
    for pos in range(5, 5 + W + 2):
        got, want = t.step(pos, q=q)
        assert off(got, want) < (1e-5 if not bf16 else 3e-3), pos
        before = want if pos == 4 + W - 1 else before
    assert off(before, want) > 0.2  # it did show while it was inside


# ------------------------------------------------------------------ whole models
@pytest.fixture(scope="module")
def folder(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            cfg, w = CONFIGS[name], weights(CONFIGS[name], 100 + len(name))
            made[name] = (write_folder(str(tmp_path_factory.mktemp(name)), cfg, w), cfg, w)
        return made[name]
    return get


def tokens(cfg, n, seed=0):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n)


LIMIT = {"f32": 2e-5, "bf16": 4e-2}


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_layers_and_logits(folder, name, dtype):
    path, cfg, w = folder(name)
    ids, streams = tokens(cfg, 150), []
    want = L.forward(cfg, w, ids, layers_out=streams)
    m = load_model(path, weight_dtype=dtype, max_seq_len=400)
    s = m.session(max_ctx=200)
    got, res = s.feed(ids, want=range(150), want_residuals=True)
    for i, (a, b) in enumerate(zip(res, streams)):
        assert off(a, b) < LIMIT[dtype], i
    rows = [off(g, x) for g, x in zip(got[0], want)]
    assert max(rows) < 2.5 * LIMIT[dtype] and off(got[0], want) < LIMIT[dtype]
    assert off(m.forward(ids), want[-1]) < 2.5 * LIMIT[dtype]
    assert off(m.forward_all(ids[:70]), want[:70]) < LIMIT[dtype]
    assert m.num_parameters() == sum(a.size for a in w.values()) and m.name() == cfg["architecture"]


@pytest.mark.parametrize("name", BOFIRAX)
def test_the_limit_would_show_a_mistake(folder, name):
    """Mistakes planted in the oracle move its logits well beyond the limits of these tests."""
    _, cfg, w = folder(name)
    ids = tokens(cfg, 150)
    right = L.forward(cfg, w, ids)
    for i, layer in enumerate(cfg["layers"]):
        m = layer["mixer"]
        changed = json.loads(json.dumps(cfg))
        if layer["type"] == "latent_attention" and "mask" in m:
            changed["layers"][i]["mixer"]["mask"]["size"] += 1
            assert off(L.forward(changed, w, ids)[100:], right[100:]) > 20 * LIMIT["f32"]
        if layer["type"].startswith("delta") and m["heads"] > 1:
            swapped = dict(w)
            swapped[f"l{i}.mix.A_log"] = w[f"l{i}.mix.A_log"][::-1]
            assert off(L.forward(cfg, swapped, ids), right) > 20 * LIMIT["f32"]
        without = dict(w)
        without[f"l{i}.ls1"] = np.ones_like(w[f"l{i}.ls1"])
        assert off(L.forward(cfg, without, ids), right) > LIMIT["bf16"]


@pytest.mark.parametrize("name", ZEKILIX)
def test_the_limit_would_show_a_mistake_in_these(folder, name):
    _, cfg, w = folder(name)
    ids = tokens(cfg, 150)
    right = L.forward(cfg, w, ids)

    def moved(change=None, w2=None, at=slice(None), by=20 * LIMIT["f32"]):
        c = json.loads(json.dumps(cfg))
        if change:
            change(c)
        assert off(L.forward(c, w2 or w, ids)[at], right[at]) > by

    moved(lambda c: c.update(residual_mult=1.01 * c["residual_mult"]))
    moved(lambda c: c.update(logit_softcap=1.01 * c["logit_softcap"]))
    moved(lambda c: c["embedding"].update(scale=1.01 * c["embedding"]["scale"]))
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{L.tensors_of(cfg, i)}."
        if "mask" in m:
            moved(lambda c: c["layers"][i]["mixer"]["mask"].update(size=m["mask"]["size"] + 1), at=slice(100, None))
        if "kv_heads" in m:
            moved(lambda c: c["layers"][i]["mixer"].update(scale=1.02 * m["scale"]) if m.get("mask") != {"size": 1} else
                  c.update(residual_mult=0.5 * c["residual_mult"]))
        if "gate_cap" in m:
            moved(lambda c: c["layers"][i]["mixer"].update(gate_cap=1.1 * m["gate_cap"]))
        if layer["mlp"]:
            moved(lambda c: c["layers"][i]["mlp"].update(limit=1.1 * layer["mlp"]["limit"]))
        if cfg["streams"] > 1:
            hc = p + ("hc2" if layer["mlp"] else "hc1")
            moved(w2={**w, hc + ".mix": w[hc + ".mix"].T})
            if i < len(cfg["layers"]) - 1:  # (behind the last one only their sum counts)
                moved(w2={**w, hc + ".out": w[hc + ".out"][::-1]})
            if i or layer["mlp"]:  # (the streams are equal in front of the first sublayer)
                moved(w2={**w, hc + ".in": w[hc + ".in"][::-1]})


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_decoding_and_portions(folder, name, dtype):
    """Token by token from the start; a prompt and then token by token; portions of changing size down to
    two tokens: the same logits at every position."""
    path, cfg, w = folder(name)
    ids = tokens(cfg, 120, 1)
    want = L.forward(cfg, w, ids)
    m = load_model(path, weight_dtype=dtype)
    for cuts in ([1] * 120, [60] + [1] * 60, [2, 3, 1, 17, 2, 33, 2, 1, 1, 40, 2, 16], [119, 1]):
        s, pos, worst = m.session(max_ctx=128), 0, 0.0
        for c in cuts:
            part = ids[pos:pos + c]
            got = s.decode(part) if c == 1 and pos else s.feed(part, want=range(c))[0]
            for j in range(c):
                worst = max(worst, off(got[j], want[pos + j]))
            pos += c
        assert pos == 120 == s.position and worst < 2.5 * LIMIT[dtype], cuts[:3]
        s.close()


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
@pytest.mark.parametrize("name", ["mixed", "odd", "wide", "hyper", "hyper_odd", "hyper_wide"])
def test_batches_and_reused_sessions(folder, name, dtype):
    path, cfg, w = folder(name)
    m = load_model(path, weight_dtype=dtype, max_batch=3)
    ids = np.stack([tokens(cfg, 90, 10 + b) for b in range(3)])
    want = [L.forward(cfg, w, row) for row in ids]
    s = m.session(batch=3, max_ctx=100)
    for _ in range(2):  # the second time in a session that has been used
        first = s.prefill(ids[:, :50])
        more = s.feed(ids[:, 50:70], want=[0, 19])
        last = [s.decode(ids[:, i]) for i in range(70, 90)]
        for b in range(3):
            assert off(first[b], want[b][49]) < 2.5 * LIMIT[dtype]
            assert off(more[b], want[b][[50, 69]]) < 2.5 * LIMIT[dtype]
            assert max(off(g[b], want[b][70 + i]) for i, g in enumerate(last)) < 2.5 * LIMIT[dtype]
        s.reset()
        assert s.position == 0
        s.feed(ids[:, ::-1][:, :77])  # something else in between
        s.reset()
    # alone, in another session of the same model while the first one lives
    one = m.session(max_ctx=100)
    assert off(one.feed(ids[1], want=range(90))[0], want[1]) < LIMIT[dtype]


def oracle_greedy(cfg, w, ids, n):
    ids, out, margin = list(ids), [], np.inf
    for _ in range(n):
        z = L.forward(cfg, w, ids)[-1]
        top = np.sort(z)[-2:]
        margin = min(margin, top[1] - top[0])
        out.append(int(z.argmax()))
        ids.append(out[-1])
    return out, margin


@pytest.mark.parametrize("name", ["mixed", "hyper", "hyper_odd"])
def test_greedy_generation(folder, name):
    """The plugin's own generation (prompt pass, then graph-replayed steps past the windows) against greedy
    decoding of the oracle; graph replay against kernel-by-kernel launches, replayed again after a reset."""
    path, cfg, w = folder(name)
    ids = tokens(cfg, 20, 2)
    want, margin = oracle_greedy(cfg, w, ids, 40)
    assert margin > 1e-4  # (no step hangs on a rounding)
    m = load_model(path, weight_dtype="f32", max_seq_len=256)
    assert m.generate(ids, BasicGenerationConfig(max_length=40, temperature=0.0)) == want
    for dtype in ("f32", "bf16"):
        m = load_model(path, weight_dtype=dtype, max_seq_len=256, max_batch=2)
        for batch in (1, 2):
            s = m.session(batch=batch, max_ctx=200)
            runs = []
            for graph in (True, False, True):
                s.set_graph(graph)
                s.reset()
                tok = s.prefill(np.tile(ids, (batch, 1))).argmax(-1)
                runs.append(np.concatenate([s.decode_greedy(tok, 70), s.decode_greedy(tok, 50)], axis=1))
            assert np.array_equal(runs[0], runs[1]) and np.array_equal(runs[0], runs[2])
            assert dtype != "f32" or list(runs[0][0, :39]) == want[1:]
            s.close()


@pytest.mark.parametrize("name", ["wide", "hyper_wide"])
def test_sampling_is_reproducible(folder, name):
    path, cfg, _ = folder(name)
    m = load_model(path, max_seq_len=128)
    ids, how = tokens(cfg, 12, 3), BasicGenerationConfig(max_length=30, temperature=12.0, top_k=20, top_p=0.9)
    a, b, c = (m.generate(ids, how, seed=s) for s in (1, 1, 2))
    assert a == b != c and len(a) == 30 and max(a) < cfg["vocab"]


LONG = {"Bofirax": config(48, 60, [delta(2, 1, 16, 24, 4), latent(2, 16, 16, 24, 32, 19, ff=48), delta(2, 2, 12, 16, 3)]),
        "Zekilix": hyper_config(48, 60, [memory(2, 16, 24), shared_kv(4, 2, 16, 19, ff=48), memory(3, 12, 16, cap=5.0)], 3)}


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
@pytest.mark.parametrize("design", sorted(LONG))
def test_long_decoding(design, dtype, tmp_path):
    """Hundreds of decoded tokens: the rings come round many times, the state keeps going."""
    cfg = LONG[design]
    w = weights(cfg, 9)
    ids = tokens(cfg, 700, 4)
    want = L.forward(cfg, w, ids)
    s = load_model(write_folder(str(tmp_path), cfg, w), weight_dtype=dtype).session(max_ctx=700)
    s.prefill(ids[:100], want_logits=False)
    errs = [off(s.decode(ids[i:i + 1])[0], want[i]) for i in range(100, 700)]
    assert max(errs) < 4 * LIMIT[dtype] and np.mean(errs[-100:]) < 2 * LIMIT[dtype]
    with pytest.raises(ProcessingError, match="out of range"):
        s.decode(ids[:1])


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
@pytest.mark.parametrize("name", ["mixed", "hyper"])
def test_trace_program_on_a_model(folder, tmp_path, name, dtype):
    path, cfg, w = folder(name)
    a, b = tokens(cfg, 40, 5), tokens(cfg, 31, 6)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:30].tolist(), "want": [3, 29]}], "end": []}]
    steps += [{"step": 1 + i, "entries": [{"id": "a", "tokens": [int(a[30 + i])], "want": [0]}], "end": ["a"] if i == 9 else []}
              for i in range(10)]
    steps += [{"step": 11, "entries": [{"id": "b", "tokens": b[:2].tolist(), "want": [1]}], "end": []},
              {"step": 12, "entries": [{"id": "b", "tokens": b[2:].tolist(), "want": [28, 0]}], "end": ["b"]}]
    m = load_model(path, weight_dtype=trace.DTYPES[dtype], max_seq_len=40)
    said = []
    trace.run(m, str(tmp_path), 40, [json.dumps(s) for s in steps], said.append)
    assert said == [f"done {i}" for i in range(13)]
    lim = 2.5 * LIMIT[trace.DTYPES[dtype]]
    rows = lambda n: np.fromfile(tmp_path / f"{n}.f32", "<f4").reshape(-1, cfg["vocab"])
    wa, wb = L.forward(cfg, w, a), L.forward(cfg, w, b)
    assert off(rows(0), wa[[3, 29]]) < lim and off(rows(11), wb[[1]]) < lim and off(rows(12), wb[[30, 2]]) < lim
    assert max(off(rows(1 + i), wa[[30 + i]]) for i in range(10)) < lim


def test_synthetic_models_and_refusals():
    cfg = CONFIGS["wide"]
    b = PLUGINS["layered_model"].create_builder()
    m = b.build(LayeredConfig(cfg, max_seq_len=64), seed=3)
    z = m.session(max_ctx=64).feed(tokens(cfg, 60), want=[0, 59])
    assert np.isfinite(z).all() and z.std() > 0
    ms, n, by = m.session(max_ctx=64).time_decode_matmuls(2)
    assert ms > 0 and n == 2 * (3 * 2 + 1 + 4 + 1) and by > 0
    s = m.session(max_ctx=64)
    with pytest.raises(ProcessingError, match="Token ID"):
        s.feed([cfg["vocab"]], want=[0])
    with pytest.raises(ProcessingError, match="Row 2 out of range"):
        s.feed([1, 2], want=[2])
    with pytest.raises(ProcessingError, match="Sequence length"):
        s.feed(np.zeros(65, dtype=np.uint64))
    with pytest.raises(ProcessingError, match="no place"):
        m.write_to("x")
    with pytest.raises(ProcessingError, match="Batch 2 out of range"):
        m.session(batch=2)


def test_feed_on_the_transformer(orc):
    """The chosen rows and the streams behind the blocks work for the other family as well."""
    from coeus_amd import Transformer250MConfig, TransformerModelPlugin
    cfg = Transformer250MConfig(hidden_dim=64, num_layers=3, num_heads=4, intermediate_dim=96, vocab_size=211, max_seq_len=48,
                                norm_scope="token")
    m = TransformerModelPlugin().create_builder().build(cfg, seed=5)
    ids = np.arange(40) * 5 % 211
    every = m.forward_all(ids)
    s = m.session(max_ctx=48)
    got, res = s.feed(ids[:25], want=[0, 24, 7], want_residuals=True)
    more = s.feed(ids[25:], want=[14])
    assert off(got[0], every[[0, 24, 7]]) < 1e-5 and off(more[0], every[[39]]) < 1e-5
    assert res.shape == (3, 25, 64) and np.isfinite(res).all() and off(res[0], res[1]) > 1e-3
