"""Small layered models for the tests: configurations, random weights, and a writer of the folder that
coeus_model_load reads."""
import copy
import json
import os
import struct

import numpy as np


def delta(heads, kv_heads, dim, vdim, conv, ff=None, kind="delta"):
    return {"type": kind, "mixer": dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv),
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def latent(heads, dim, vdim, q_rank, kv_rank, window, scale=None, ff=None):
    m = dict(heads=heads, dim=dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, scale=scale or dim ** -0.5)
    if window is not None:
        m["mask"] = {"size": window}
    return {"type": "latent_attention", "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def memory(heads, dim, vdim, cap=9.0, ff=None, limit=1.5, kind="mlstm"):
    return {"type": kind, "mixer": dict(heads=heads, dim=dim, vdim=vdim, gate_cap=cap),
            "mlp": None if ff is None else {"kind": "dense", "ff": ff, "limit": limit}}


def shared_kv(heads, kv_heads, dim, window, scale=None, ff=None, limit=1.5, kind="attention"):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=scale or dim ** -0.5)
    if window is not None:
        m["mask"] = {"size": window}
    return {"type": kind, "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff, "limit": limit}}


def again(layers, i):
    """Another layer with layer i's tensors."""
    return {**copy.deepcopy(layers[i]), "weights_of": i}


def hyper_config(width, vocab, layers, streams, eps=1e-5, mult=0.45, softcap=8.0, scale=3.5):
    return {"architecture": "Zekilix", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers, "streams": streams,
            "residual_mult": mult, "logit_softcap": softcap, "embedding": {"scale": scale}}


def hyper_shared():
    ls = [shared_kv(6, 3, 24, 17, ff=72), memory(4, 16, 24), memory(2, 40, 48, cap=4.0, ff=64, limit=0.7)]
    ls += [again(ls, 1), again(ls, 0), shared_kv(4, 4, 32, 33, kind="attention_2")]
    return ls + [again(ls, 2), again(ls, 3)]  # (the last one's tensors are another's in turn)


def config(width, vocab, layers, eps=1e-5):
    return {"architecture": "Bofirax", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers}


# name -> configuration: orders, sizes and windows that differ from each other, some of them not multiples of
# what the kernels move at once, a window of one, layers with and without feed-forward
CONFIGS = {
    "mixed": config(96, 131, [latent(3, 24, 16, 40, 48, 17, ff=72), delta(4, 2, 16, 32, 4), delta(2, 2, 40, 48, 2, ff=64),
                              latent(2, 32, 64, 32, 64, 33)], eps=1e-6),
    "odd": config(58, 89, [delta(3, 1, 10, 7, 5, ff=30), latent(3, 12, 9, 21, 19, 5, scale=0.4), delta(2, 1, 9, 20, 1)]),
    "wide": config(128, 200, [delta(4, 4, 64, 128, 4, ff=160), delta(2, 1, 128, 64, 3, kind="delta_2"),
                              latent(4, 64, 64, 64, 128, 64, ff=128)], eps=1e-4),
    "one": config(64, 77, [latent(2, 16, 24, 24, 32, 1, ff=40), delta(2, 2, 8, 8, 2, ff=24)]),
    "unbounded": config(64, 96, [delta(2, 1, 24, 16, 3), latent(2, 32, 32, 32, 96, None, ff=64)]),
    "hyper": hyper_config(96, 131, hyper_shared(), 2, eps=1e-6),
    "hyper_odd": hyper_config(58, 89, [memory(3, 10, 7, ff=30), shared_kv(3, 1, 9, 5, scale=0.4, ff=22), memory(1, 9, 20, cap=2.5)], 5,
                              mult=1.3, softcap=4.0, scale=0.7),
    "hyper_wide": hyper_config(128, 200, [memory(4, 64, 128, ff=160), shared_kv(8, 2, 64, 64, ff=128), memory(2, 128, 64, cap=20.0)],
                               4, eps=1e-4, mult=0.6),
    "hyper_one": hyper_config(64, 77, [shared_kv(2, 2, 16, 1, ff=40), memory(2, 8, 8, ff=24)], 1, mult=1.0, scale=1.0),
    "hyper_unbounded": hyper_config(64, 96, [memory(2, 24, 16), shared_kv(5, 1, 40, None, ff=64)], 3, softcap=9.0),
}
BOFIRAX = sorted(n for n, c in CONFIGS.items() if c["architecture"] == "Bofirax")
ZEKILIX = sorted(n for n, c in CONFIGS.items() if c["architecture"] == "Zekilix")


def bf16_round(a):
    u = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32).astype(np.uint64)
    u = ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint32) << 16
    return u.view(np.float32).reshape(np.shape(a))


def shapes(cfg):
    W, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"])}
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}."
        if layer.get("weights_of") is not None:
            continue
        if cfg["architecture"] == "Zekilix":
            out.update(hyper_layer_shapes(cfg, layer, p))
            continue
        if layer["type"].startswith("delta"):
            qk, v = m["kv_heads"] * m["dim"], m["heads"] * m["vdim"]
            for t, n in (("q", qk), ("k", qk), ("v", v)):
                out[p + f"mix.{t}"], out[p + f"mix.{t}.conv"] = (n, W), (n, m["conv"])
            out.update({p + "mix.g": (v, W), p + "mix.b": (m["heads"], W), p + "mix.a": (m["heads"], W),
                        p + "mix.A_log": (m["heads"],), p + "mix.dt_bias": (m["heads"],), p + "mix.norm": (m["vdim"],),
                        p + "mix.o": (W, v)})
        else:
            out.update({p + "mix.dq": (m["q_rank"], W), p + "mix.dq.norm": (m["q_rank"],),
                        p + "mix.uq": (m["heads"] * m["dim"], m["q_rank"]), p + "mix.dkv": (m["kv_rank"], W),
                        p + "mix.dkv.norm": (m["kv_rank"],), p + "mix.uk": (m["heads"] * m["dim"], m["kv_rank"]),
                        p + "mix.uv": (m["heads"] * m["vdim"], m["kv_rank"]), p + "mix.o": (W, m["heads"] * m["vdim"])})
        out[p + "norm1"] = out[p + "ls1"] = (W,)
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            out.update({p + "mlp.gate": (ff, W), p + "mlp.up": (ff, W), p + "mlp.down": (W, ff), p + "norm2": (W,), p + "ls2": (W,)})
    out["final.norm"] = (W,)
    if cfg["architecture"] == "Zekilix":
        out["head"] = (cfg["vocab"], W)
    return out


def hyper_layer_shapes(cfg, layer, p):
    W, s, m, out = cfg["width"], cfg["streams"], layer["mixer"], {}
    qk, v = m["heads"] * m["dim"], m["heads"] * m["vdim"]
    if layer["type"].startswith("mlstm"):
        out.update({p + f"mix.{t}": (n, W) for t, n in (("q", qk), ("k", qk), ("v", v), ("g", v), ("i", m["heads"]), ("f", m["heads"]))})
        out.update({p + "mix.i.b": (m["heads"],), p + "mix.f.b": (m["heads"],), p + "mix.norm": (v,)})
    else:
        kv = m["kv_heads"] * m["dim"]
        out.update({p + "mix.q": (qk, W), p + "mix.k": (kv, W), p + "mix.q.norm": (qk,), p + "mix.k.norm": (kv,), p + "mix.g": (v, W)})
    out[p + "mix.o"] = (W, v)
    subs = ["1"]
    if layer["mlp"] is not None:
        ff = layer["mlp"]["ff"]
        out.update({p + "mlp.gate": (ff, W), p + "mlp.up": (ff, W), p + "mlp.down": (W, ff)})
        subs.append("2")
    for q in subs:
        out.update({p + "norm" + q: (W,), p + f"hc{q}.in": (s,), p + f"hc{q}.out": (s,), p + f"hc{q}.mix": (s, s)})
    return out


def weights(cfg, seed, sharp=2.0):
    """Random weights, rounded to bf16.  Queries and keys of the attention are `sharp` times larger than
    unit variance would ask for (or their norms' weights are), so that single keys carry weight; decays and gates
    run from slow to fast."""
    rng, out = np.random.default_rng(seed), {}
    for name, shape in shapes(cfg).items():
        last = name.split(".")[-1]
        if last == "A_log":
            a = rng.uniform(-4.0, 1.0, shape)
        elif last == "dt_bias":
            a = rng.uniform(-3.0, 1.0, shape)
        elif last == "conv":
            a = rng.normal(0.0, 0.6, shape)
        elif name.endswith(".f.b"):
            a = rng.uniform(0.0, 6.0, shape)
        elif name.endswith(".i.b"):
            a = rng.uniform(-4.0, 3.0, shape)
        elif name.endswith("hc1.mix") or name.endswith("hc2.mix"):
            a = 0.8 * np.eye(shape[0]) + rng.normal(0.0, 0.25, shape)
        elif len(shape) == 1:
            a = rng.uniform(0.5, 1.5, shape)
            if name.endswith(("mix.q.norm", "mix.k.norm")):
                a = a * sharp
        else:
            a = rng.normal(0.0, 1.0, shape) / np.sqrt(shape[1] if last != "embed" else 1.0)
            if last in ("uq", "uk"):
                a = a * sharp
            if last == "head":
                a = 3.0 * a  # (so that the cap on the logits shows)
        out[name] = bf16_round(a)
    return out


def write_folder(path, cfg, w, dtype="BF16"):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    head, blobs, off = {}, [], 0
    for name, a in w.items():
        a = np.ascontiguousarray(a, dtype=np.float32)
        data = a.tobytes() if dtype == "F32" else (a.view(np.uint32) >> 16).astype(np.uint16).tobytes()
        head[name] = {"dtype": dtype, "shape": list(a.shape), "data_offsets": [off, off + len(data)]}
        blobs.append(data)
        off += len(data)
    text = json.dumps(head).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(text)) + text + b"".join(blobs))
    return path
