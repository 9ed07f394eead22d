"""Layered models without a device: the oracle's mechanisms against what they must reduce to, the
configuration and weight-file readers of the library, the trace program's argument handling."""
import copy
import ctypes as C
import json
import os
import struct

import numpy as np
import pytest

from coeus_amd import PLUGINS, ConfigError, LayeredConfig, ProcessingError, _lib, load_model, trace
from coeus_amd.plugin import _check
from layered_util import CONFIGS, memory, hyper_config, shapes, weights, write_folder
from oracle import layered as L


# ------------------------------------------------------------------ oracle
def test_delta_rule_reduces_to_known_forms():
    rng = np.random.default_rng(1)
    T, d, e = 9, 4, 3
    k = np.eye(d)[rng.integers(0, d, T)]
    q, v = rng.normal(size=(T, d)), rng.normal(size=(T, e))
    # unit keys, beta = 1, no decay: the state is a table that the last write of a key wins
    out, S = L.delta_rule(q, k, v, np.ones(T), np.ones(T))
    table = np.zeros((d, e))
    for t in range(T):
        table[k[t].argmax()] = v[t]
        assert np.allclose(out[t], q[t] @ table)
    assert np.allclose(S, table)
    # full decay: only the current token is seen
    out, _ = L.delta_rule(q, k, v, np.full(T, 0.5), np.zeros(T))
    assert np.allclose(out, 0.5 * np.sum(q * k, -1, keepdims=True) * v)
    # cut anywhere, the state carries over
    b, g = rng.uniform(size=T), rng.uniform(size=T)
    kk = L.unit(rng.normal(size=(T, d)))
    whole, S = L.delta_rule(q, kk, v, b, g)
    a1, s1 = L.delta_rule(q[:4], kk[:4], v[:4], b[:4], g[:4])
    a2, s2 = L.delta_rule(q[4:], kk[4:], v[4:], b[4:], g[4:], s1)
    assert np.allclose(whole, np.concatenate([a1, a2])) and np.allclose(S, s2)


def test_short_conv_is_causal_and_ordered():
    x, taps = np.zeros((6, 1)), np.array([[0.25, -2.0, 3.0]])
    x[2] = 1.0
    pre = np.array([0, 0, 3.0, -2.0, 0.25, 0])
    assert np.allclose(L.short_conv(x, taps)[:, 0], pre / (1 + np.exp(-pre)))


def test_window_edges_of_the_attention():
    """A key that outweighs all others is seen at distance window - 1 and not at distance window."""
    T, W = 12, 4
    q, k, v = np.ones((T, 1)), np.zeros((T, 1)), np.zeros((T, 1))
    k[3], v[3] = 50.0, 1.0
    out = L.masked_attention(q, k, v, 1.0, W)[:, 0]
    assert np.allclose(out, [0, 0, 0, 1, 1, 1, 1, 0, 0, 0, 0, 0])
    assert np.allclose(L.masked_attention(q, k, v, 1.0, None)[3:, 0], 1.0)


def test_matrix_memory_reduces_to_known_forms():
    rng = np.random.default_rng(4)
    T, d, e = 9, 4, 3
    q, k, v = rng.normal(size=(T, d)), rng.normal(size=(T, d)), rng.normal(size=(T, e))
    # nothing forgotten, unit input gates (their logarithm 0 is the maximum's start): linear attention over the
    # normaliser, whose floor is 1
    out, (S, n, m) = L.matrix_memory(q, k, v, np.zeros(T), np.zeros(T))
    for t in range(T):
        s = k[:t + 1] @ q[t]
        assert np.allclose(out[t], s @ v[:t + 1] / (max(abs(s.sum()), 1.0) + 1e-6))
    assert np.allclose(S, k.T @ v) and np.allclose(n, k.sum(0)) and m == 0
    # the maximum only changes how numbers are held: against the recurrence without it, with the floor e^0
    li, lf = rng.normal(size=T) * 2, L.log_sigmoid(rng.normal(size=T))
    out, (S, n, m) = L.matrix_memory(q, k, v, li, lf)
    S1, n1 = np.zeros((d, e)), np.zeros(d)
    for t in range(T):
        S1, n1 = np.exp(lf[t]) * S1 + np.exp(li[t]) * np.outer(k[t], v[t]), np.exp(lf[t]) * n1 + np.exp(li[t]) * k[t]
        assert np.allclose(out[t], S1.T @ q[t] / max(abs(n1 @ q[t]), 1.0), rtol=1e-4)
    assert np.allclose(S * np.exp(m), S1) and np.allclose(n * np.exp(m), n1)
    # cut anywhere, the state carries over
    a1, s1 = L.matrix_memory(q[:4], k[:4], v[:4], li[:4], lf[:4])
    a2, s2 = L.matrix_memory(q[4:], k[4:], v[4:], li[4:], lf[4:], s1)
    assert np.allclose(np.concatenate([a1, a2]), out) and np.allclose(s2[0], S)


def test_distance_bias():
    """A score's bias is slope times distance, slopes falling by powers from 2^(-8/H) to 2^-8."""
    assert np.allclose(L.distance_slopes(4), [2.0 ** -2, 2.0 ** -4, 2.0 ** -6, 2.0 ** -8])
    q, k, v = np.zeros((3, 1)), np.zeros((3, 1)), np.array([[1.0], [2.0], [4.0]])
    w = np.exp([-1.0, -0.5, 0.0])
    assert np.allclose(L.biased_attention(q, k, v, 1.0, None, 0.5)[2], w @ v / w.sum())
    assert np.allclose(L.biased_attention(q, k, v, 1.0, 2, 0.5)[2], w[1:] @ v[1:] / w[1:].sum())


def test_hyper_connections_reduce_to_known_forms():
    rng = np.random.default_rng(6)
    xs, y = rng.normal(size=(3, 4, 5)), rng.normal(size=(4, 5))
    # from first: stream 0 goes to stream 2 alone, nothing else anywhere
    mix = np.zeros((3, 3))
    mix[0, 2] = 2.0
    new = L.hyper_write(xs, mix, np.array([0.0, 1.0, 0.0]), y, 0.5)
    assert np.allclose(new[0], 0) and np.allclose(new[1], 0.5 * y) and np.allclose(new[2], 2.0 * xs[0])
    # one stream with all weights 1 is the plain residual sum
    assert np.allclose(L.hyper_write(xs[:1], np.eye(1), np.ones(1), y, 0.5)[0], xs[0] + 0.5 * y)
    assert np.allclose(L.hyper_read(xs, np.array([1.0, -1.0, 0.5])), xs[0] - xs[1] + 0.5 * xs[2])


def test_clamped_gate():
    W = {"m.gate": np.array([[1.0]]), "m.up": np.array([[-1.0]]), "m.down": np.array([[1.0]])}
    x = np.array([[0.5], [9.0], [-9.0]])
    g, u = np.array([0.5, 2.0, -9.0]), np.array([-0.5, -2.0, 2.0])
    assert np.allclose(L.clamped_ff(x, W, "m", 2.0)[:, 0], g / (1 + np.exp(-1.702 * g)) * (u + 1))


# ------------------------------------------------------------------ configuration
def check_text(text):
    n = C.c_uint64()
    _check(_lib.load().coeus_layered_config_check(text, len(text), C.byref(n)))
    return n.value


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_parameter_counts(name):
    cfg = CONFIGS[name]
    want = sum(int(np.prod(s)) for s in shapes(cfg).values())
    assert LayeredConfig(cfg).num_parameters() == want == check_text(json.dumps(cfg, indent=3).encode())


def broken(path, value, name="mixed"):
    cfg = copy.deepcopy(CONFIGS[name])
    at = cfg
    for p in path[:-1]:
        at = at[p]
    if value is None:
        del at[path[-1]]
    else:
        at[path[-1]] = value
    return json.dumps(cfg).encode()


@pytest.mark.parametrize("path,value,message", [
    (("architecture",), "Nothing", "unknown architecture"),
    (("architecture",), None, "architecture"),
    (("width",), 0, "width"),
    (("width",), 2.5, "width"),
    (("vocab",), "12", "vocab"),
    (("norm",), None, "norm"),
    (("norm", "eps"), None, "norm.eps"),
    (("layers",), [], "layers"),
    (("layers", 1, "type"), "delta_x", "unknown layer type"),
    (("layers", 1, "type"), "conv", "unknown layer type"),
    (("layers", 1, "mixer", "kv_heads"), 3, "multiple of kv_heads"),
    (("layers", 1, "mixer", "conv"), None, "conv"),
    (("layers", 1, "mixer", "dim"), 300, "more than 256"),
    (("layers", 0, "mixer", "kv_rank"), None, "kv_rank"),
    (("layers", 0, "mixer", "scale"), None, "scale"),
    (("layers", 0, "mixer", "mask"), {"size": 0}, "mask.size"),
    (("layers", 0, "mlp", "kind"), "experts", "unknown feed-forward"),
    (("layers", 0, "mlp", "ff"), -1, "mlp.ff"),
])
def test_bad_configurations_are_named(path, value, message):
    with pytest.raises(ConfigError, match=message):
        check_text(broken(path, value))


@pytest.mark.parametrize("path,value,message", [
    (("streams",), None, "streams"),
    (("streams",), 9, "streams"),
    (("streams",), 1.5, "streams"),
    (("residual_mult",), None, "residual_mult"),
    (("logit_softcap",), 0, "logit_softcap"),
    (("embedding",), None, "embedding"),
    (("embedding", "scale"), "1", "embedding.scale"),
    (("layers", 0, "type"), "delta", "unknown layer type"),
    (("layers", 0, "mixer", "vdim"), 25, "vdim"),
    (("layers", 0, "mixer", "kv_heads"), 4, "multiple of kv_heads"),
    (("layers", 0, "mixer", "scale"), None, "scale"),
    (("layers", 0, "mlp", "limit"), None, "mlp.limit"),
    (("layers", 1, "mixer", "gate_cap"), None, "gate_cap"),
    (("layers", 1, "mixer", "gate_cap"), -1.0, "gate_cap"),
    (("layers", 1, "mixer", "dim"), 513, "more than 512"),
    (("layers", 3, "weights_of"), 8, "number of a layer"),
    (("layers", 3, "weights_of"), 0.5, "number of a layer"),
    (("layers", 3, "weights_of"), 3, "from itself"),
    (("layers", 3, "weights_of"), 2, "the two layers differ"),
    (("layers", 1, "weights_of"), 3, "no layer of this chain"),
    (("layers", 4, "mixer", "mask", "size"), 18, "the two layers differ"),
    (("layers", 6, "mlp", "limit"), 0.8, "the two layers differ"),
])
def test_bad_hyper_configurations_are_named(path, value, message):
    with pytest.raises(ConfigError, match=message):
        check_text(broken(path, value, "hyper"))


def test_layers_that_share_tensors():
    """A layer without tensors of its own adds none; forward references and chains resolve."""
    a = memory(2, 8, 12, ff=24)
    one = LayeredConfig(hyper_config(32, 50, [a], 2)).num_parameters()
    assert LayeredConfig(hyper_config(32, 50, [{**a, "weights_of": 2}, {**a, "weights_of": 0}, a], 2)).num_parameters() == one
    shared = hyper_config(32, 50, [a, {**a, "weights_of": 0}, {**a, "weights_of": 1}], 2)
    assert LayeredConfig(shared).num_parameters() == one == sum(int(np.prod(s)) for s in shapes(shared).values())


@pytest.mark.parametrize("text", [b"", b"{", b"[1,]", b'{"a": 01}', b'{"a": 1} x', b'"\\ud800"', b'{"a" 1}', b"nul",
                                  b'{"a": .5}', b"[" * 200 + b"]" * 200, b'"\x01"'])
def test_text_that_is_not_json(text):
    with pytest.raises(ConfigError, match="not JSON"):
        check_text(text)


def test_json_escapes_and_repeated_keys():
    text = json.dumps(CONFIGS["one"]).replace('"Bofirax"', '"\\u0042of\\u0069rax"').replace('"width": 64', '"width": 9, "width": 64')
    assert check_text(text.encode()) == LayeredConfig(CONFIGS["one"]).num_parameters()


def test_layer_types_may_carry_a_number():
    assert check_text(broken(("layers", 1, "type"), "delta_7")) == LayeredConfig(CONFIGS["mixed"]).num_parameters()


# ------------------------------------------------------------------ weight files
def check_folder(path):
    n = C.c_uint64()
    _check(_lib.load().coeus_layered_check(os.fsencode(path), C.byref(n)))
    return n.value


def test_weight_folder_is_checked(tmp_path):
    cfg = CONFIGS["mixed"]
    w = weights(cfg, 3)
    path = write_folder(str(tmp_path / "m"), cfg, w)
    assert check_folder(path) == LayeredConfig(cfg).num_parameters()
    assert check_folder(write_folder(str(tmp_path / "f"), cfg, w, dtype="F32")) == LayeredConfig(cfg).num_parameters()
    missing = dict(w)
    del missing["l1.mix.dt_bias"]
    with pytest.raises(ProcessingError, match="no tensor l1.mix.dt_bias"):
        check_folder(write_folder(str(tmp_path / "a"), cfg, missing))
    wrong = dict(w)
    wrong["l0.mix.uk"] = wrong["l0.mix.uk"].T
    with pytest.raises(ProcessingError, match="l0.mix.uk does not have the shape"):
        check_folder(write_folder(str(tmp_path / "b"), cfg, wrong))
    with pytest.raises(ProcessingError, match="Failed to open"):
        check_folder(str(tmp_path / "nothing"))


def test_damaged_weight_files(tmp_path):
    cfg = CONFIGS["one"]
    path = write_folder(str(tmp_path / "m"), cfg, weights(cfg, 4))
    file = os.path.join(path, "model.safetensors")
    good = open(file, "rb").read()
    n = struct.unpack("<Q", good[:8])[0]
    head = json.loads(good[8:8 + n])

    def rewrite(h, tail=good[8 + n:]):
        text = json.dumps(h).encode()
        open(file, "wb").write(struct.pack("<Q", len(text)) + text + tail)

    def refused(message):
        with pytest.raises(ProcessingError, match=message):
            check_folder(path)

    for cut in (0, 7, 8, 8 + n // 2):
        open(file, "wb").write(good[:cut])
        refused("too short|does not fit|bad header")
    open(file, "wb").write(struct.pack("<Q", 1 << 63) + good[8:])
    refused("does not fit")
    open(file, "wb").write(good[:-2])  # the last tensor's data ends behind the file
    refused("bad entry")
    for key, value in (("data_offsets", [0, 1 << 60]), ("data_offsets", [8, 4]), ("data_offsets", [0]), ("dtype", 3),
                       ("shape", [1 << 40, 1 << 40]), ("shape", [-1]), ("dtype", "Q3")):
        h = copy.deepcopy(head)
        h["embed"][key] = value
        rewrite(h)
        refused("bad entry|do not agree")
    rewrite({**head, "__metadata__": {"format": "pt"}})
    assert check_folder(path) == LayeredConfig(cfg).num_parameters()


# ------------------------------------------------------------------ registry, options, trace program
def test_registry_and_options():
    assert set(PLUGINS) == {"transformer_model", "layered_model"}
    p = PLUGINS["layered_model"]
    assert p.id() == "layered_model" and {"gated_delta_rule", "matrix_memory", "hyper_connections"} <= set(p.capabilities())
    with pytest.raises(ConfigError, match="weight_dtype"):
        LayeredConfig(CONFIGS["one"], weight_dtype="q4_0").options()
    with pytest.raises(ConfigError, match="at least 1"):
        LayeredConfig(CONFIGS["one"], max_batch=0).options()
    with pytest.raises(ConfigError):
        load_model(os.path.dirname(os.path.abspath(__file__)))  # a folder without config.json


def test_trace_arguments(capsys):
    for argv in ([], ["--model", "x", "--dtype", "float16", "--out", "y", "--max-tokens", "3"],
                 ["--model", "x", "--dtype", "float32", "--out", "y", "--max-tokens", "0"]):
        with pytest.raises(SystemExit) as e:
            trace.main(argv)
        assert e.value.code == 2
    capsys.readouterr()


class FakeSession:
    """Records what a trace feeds; the logits of a token are its id and its position."""

    def __init__(self):
        self.fed, self.resets = [], 0

    @property
    def position(self):
        return len(self.fed)

    def feed(self, ids, want):
        base = len(self.fed)
        self.fed += [int(i) for i in ids.ravel()]
        return np.array([[[ids.ravel()[w], base + int(w)] for w in want]], dtype=np.float32).reshape(1, len(want), 2)

    def decode(self, ids):
        self.fed.append(int(ids[0]))
        return np.array([[ids[0], len(self.fed) - 1]], dtype=np.float32)

    def reset(self):
        self.fed, self.resets = [], self.resets + 1


def test_trace_steps(tmp_path):
    made = []

    class Model:
        def session(self, batch, max_ctx):
            assert (batch, max_ctx) == (1, 50)
            made.append(FakeSession())
            return made[-1]

    lines = [json.dumps(s) for s in (
        {"step": 0, "entries": [{"id": "a", "tokens": [5, 6, 7], "want": [2, 0]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": [8], "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": [9], "want": [0]}], "end": ["a"]},
        {"step": 3, "entries": [{"id": "b", "tokens": [4], "want": [0]}, {"id": "c", "tokens": [3, 2], "want": [1]}], "end": ["b", "c"]})]
    said = []
    trace.run(Model(), str(tmp_path), 50, lines + ["\n"], said.append)
    assert said == ["done 0", "done 1", "done 2", "done 3"]
    rows = lambda n: np.fromfile(tmp_path / f"{n}.f32", "<f4").reshape(-1, 2).tolist()
    assert rows(0) == [[7, 2], [5, 0]] and rows(2) == [[9, 4]] and rows(3) == [[4, 0], [2, 1]]
    assert not (tmp_path / "1.f32").exists()
    assert len(made) == 2 and made[0].resets == 2  # "b" got the session that "a" gave back
