"""Small layered models for the tests: configurations, random weights, and a writer of the folder that
coeus_model_load reads."""
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
}


def bf16_round(a):
    u = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32).astype(np.uint64)
    u = ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint32) << 16
    return u.view(np.float32).reshape(np.shape(a))


def shapes(cfg):
    W, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"])}
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}."
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
    return out


def weights(cfg, seed, sharp=2.0):
    """Random weights, rounded to bf16.  Queries and keys of the attention are `sharp` times larger than
    unit variance would ask for, so that single keys carry weight; decays run from slow to fast."""
    rng, out = np.random.default_rng(seed), {}
    for name, shape in shapes(cfg).items():
        last = name.split(".")[-1]
        if last == "A_log":
            a = rng.uniform(-4.0, 1.0, shape)
        elif last == "dt_bias":
            a = rng.uniform(-3.0, 1.0, shape)
        elif last == "conv":
            a = rng.normal(0.0, 0.6, shape)
        elif len(shape) == 1:
            a = rng.uniform(0.5, 1.5, shape)
        else:
            a = rng.normal(0.0, 1.0, shape) / np.sqrt(shape[1] if last != "embed" else 1.0)
            if last in ("uq", "uk"):
                a = a * sharp
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
