"""Plain, slow restatement of the layered decoder models (test infrastructure), one function per
mechanism, token by token where the mechanism is a recurrence.  numpy only; `dtype` is the type of
every intermediate (float64 unless a caller wants otherwise).  Weights come as a dictionary
name -> array, linear weights [out, in]."""
import numpy as np

UNIT_EPS = 1e-6


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def silu(x):
    return x / (1.0 + np.exp(-x))


def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def softplus(x):
    return np.logaddexp(0.0, x)


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + UNIT_EPS)


def short_conv(x, taps):
    """x [T, C], taps [C, K]: y[t, c] = silu(sum_j taps[c, j] x[t - (K - 1) + j, c]), zeros before 0."""
    T, K = x.shape[0], taps.shape[1]
    y = np.zeros_like(x)
    for t in range(T):
        for j in range(K):
            s = t - (K - 1) + j
            if s >= 0:
                y[t] = y[t] + taps[:, j] * x[s]
    return silu(y)


def delta_rule(q, k, v, beta, decay, state=None):
    """One head.  q, k [T, d], v [T, e], beta, decay [T]; state [d, e].  Returns (o [T, e], state)."""
    S = np.zeros((q.shape[1], v.shape[1]), dtype=q.dtype) if state is None else state.copy()
    out = np.zeros_like(v)
    for t in range(q.shape[0]):
        S = decay[t] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + np.outer(k[t], u)
        out[t] = S.T @ q[t]
    return out, S


def gated_delta_mixer(x, W, p, m, eps):
    """x [T, width]; p = tensor prefix ('l0.mix'), m = the mixer's sizes."""
    H, KH, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = x.shape[0]
    q = short_conv(x @ W[p + ".q"].T, W[p + ".q.conv"]).reshape(T, KH, d)
    k = short_conv(x @ W[p + ".k"].T, W[p + ".k.conv"]).reshape(T, KH, d)
    v = short_conv(x @ W[p + ".v"].T, W[p + ".v.conv"]).reshape(T, H, e)
    q, k = unit(q) * d ** -0.5, unit(k)
    beta = sigmoid(x @ W[p + ".b"].T)
    decay = np.exp(-np.exp(W[p + ".A_log"]) * softplus(x @ W[p + ".a"].T + W[p + ".dt_bias"]))
    gate = silu(x @ W[p + ".g"].T).reshape(T, H, e)
    o = np.zeros((T, H, e), dtype=x.dtype)
    for h in range(H):
        hk = h // (H // KH)
        o[:, h], _ = delta_rule(q[:, hk], k[:, hk], v[:, h], beta[:, h], decay[:, h])
    o = rms_norm(o, W[p + ".norm"], eps) * gate
    return o.reshape(T, H * e) @ W[p + ".o"].T


def masked_attention(q, k, v, scale, window):
    """One head: q, k [T, d], v [T, e]; i sees j with 0 <= i - j < window (window None: all j <= i)."""
    T = q.shape[0]
    out = np.zeros((T, v.shape[1]), dtype=q.dtype)
    for i in range(T):
        lo = 0 if window is None else max(0, i - window + 1)
        s = k[lo:i + 1] @ q[i] * scale
        a = np.exp(s - s.max())
        out[i] = (a / a.sum()) @ v[lo:i + 1]
    return out


def latent_attention_mixer(x, W, p, m, eps):
    H, d, e, T = m["heads"], m["dim"], m["vdim"], x.shape[0]
    cq = rms_norm(x @ W[p + ".dq"].T, W[p + ".dq.norm"], eps)
    q = (cq @ W[p + ".uq"].T).reshape(T, H, d)
    c = rms_norm(x @ W[p + ".dkv"].T, W[p + ".dkv.norm"], eps)
    k = (c @ W[p + ".uk"].T).reshape(T, H, d)
    v = (c @ W[p + ".uv"].T).reshape(T, H, e)
    window = (m.get("mask") or {}).get("size")
    o = np.stack([masked_attention(q[:, h], k[:, h], v[:, h], m["scale"], window) for h in range(H)], axis=1)
    return o.reshape(T, H * e) @ W[p + ".o"].T


def dense_ff(x, W, p):
    return (silu(x @ W[p + ".gate"].T) * (x @ W[p + ".up"].T)) @ W[p + ".down"].T


# ---------------------------------------------------------------- matrix memory, hyper-connections, shared keys and values
def layer_norm(x, w, eps):
    d = x - x.mean(axis=-1, keepdims=True)
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * w


def log_sigmoid(x):
    return -softplus(-x)


def soft_cap(x, cap):
    return cap * np.tanh(x / cap)


MEMORY_FLOOR = 1e-6


def matrix_memory(q, k, v, log_in, log_forget, state=None):
    """One head.  q, k [T, d], v [T, e], gates [T]; state (S [d, e], n [d], m).  The running maximum m starts
    at 0; everything is held divided by e^m.  Returns (o [T, e], state)."""
    S, n, m = (np.zeros((q.shape[1], v.shape[1]), q.dtype), np.zeros(q.shape[1], q.dtype), q.dtype.type(0)) if state is None else state
    out = np.zeros_like(v)
    for t in range(q.shape[0]):
        top = max(log_forget[t] + m, log_in[t])
        keep, add = np.exp(log_forget[t] + m - top), np.exp(log_in[t] - top)
        S = keep * S + add * np.outer(k[t], v[t])
        n = keep * n + add * k[t]
        m = top
        out[t] = S.T @ q[t] / (max(abs(n @ q[t]), np.exp(-m)) + MEMORY_FLOOR)
    return out, (S, n, m)


def memory_mixer(x, W, p, m, eps):
    H, d, e, cap, T = m["heads"], m["dim"], m["vdim"], m["gate_cap"], x.shape[0]
    q = (x @ W[p + ".q"].T).reshape(T, H, d) * d ** -0.5
    k = (x @ W[p + ".k"].T).reshape(T, H, d)
    v = (x @ W[p + ".v"].T).reshape(T, H, e)
    log_in = soft_cap(x @ W[p + ".i"].T + W[p + ".i.b"], cap)
    log_forget = log_sigmoid(soft_cap(x @ W[p + ".f"].T + W[p + ".f.b"], cap))
    o = np.stack([matrix_memory(q[:, h], k[:, h], v[:, h], log_in[:, h], log_forget[:, h])[0] for h in range(H)], axis=1)
    o = rms_norm(o, 1.0, eps).reshape(T, H * e) * W[p + ".norm"] * sigmoid(x @ W[p + ".g"].T)
    return o @ W[p + ".o"].T


def distance_slopes(heads):
    return 2.0 ** (-8.0 * (np.arange(heads) + 1) / heads)


def biased_attention(q, k, v, scale, window, slope):
    """One head, like masked_attention; slope * (i - j) is taken off the score of key j."""
    out = np.zeros((q.shape[0], v.shape[1]), dtype=q.dtype)
    for i in range(q.shape[0]):
        lo = 0 if window is None else max(0, i - window + 1)
        s = k[lo:i + 1] @ q[i] * scale - slope * (i - np.arange(lo, i + 1))
        a = np.exp(s - s.max())
        out[i] = (a / a.sum()) @ v[lo:i + 1]
    return out


def shared_kv_attention_mixer(x, W, p, m, eps):
    """Values are the keys as projected; the norms run over the whole projection."""
    H, G, d, T = m["heads"], m["kv_heads"], m["dim"], x.shape[0]
    v = x @ W[p + ".k"].T
    q = rms_norm(x @ W[p + ".q"].T, W[p + ".q.norm"], eps).reshape(T, H, d)
    k = rms_norm(v, W[p + ".k.norm"], eps).reshape(T, G, d)
    v = v.reshape(T, G, d)
    window, slopes = (m.get("mask") or {}).get("size"), distance_slopes(H)
    o = np.stack([biased_attention(q[:, h], k[:, h // (H // G)], v[:, h // (H // G)], m["scale"], window, slopes[h])
                  for h in range(H)], axis=1).reshape(T, H * d)
    return (o * sigmoid(x @ W[p + ".g"].T)) @ W[p + ".o"].T


SIGMOID_SLOPE = 1.702


def clamped_ff(x, W, p, limit):
    g = np.minimum(x @ W[p + ".gate"].T, limit)
    u = np.clip(x @ W[p + ".up"].T, -limit, limit)
    return (g * sigmoid(SIGMOID_SLOPE * g) * (u + 1.0)) @ W[p + ".down"].T


def hyper_read(xs, w_in):
    """xs [s, T, width]: the weighted sum of the streams that a sublayer reads."""
    return np.einsum("s,stw->tw", w_in, xs)


def hyper_write(xs, mix, out, y, mult):
    """New streams from the old ones (mix[from, to]) and the sublayer's output."""
    return np.einsum("st,snw->tnw", mix, xs) + mult * out[:, None, None] * y


HYPER_MIXERS = {"mlstm": memory_mixer, "attention": shared_kv_attention_mixer}


def tensors_of(cfg, i):
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def forward_hyper(cfg, W, tokens, dtype, layers_out):
    eps, mult = dtype(cfg["norm"]["eps"]), dtype(cfg["residual_mult"])
    x = W["embed"][np.asarray(tokens, dtype=np.int64)] * dtype(cfg["embedding"]["scale"])
    xs = np.stack([x] * cfg["streams"])
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{tensors_of(cfg, i)}"
        subs = [(".hc1", ".norm1", lambda u: HYPER_MIXERS[layer["type"].split("_")[0]](u, W, p + ".mix", layer["mixer"], eps))]
        if layer["mlp"] is not None:
            subs.append((".hc2", ".norm2", lambda u: clamped_ff(u, W, p + ".mlp", layer["mlp"]["limit"])))
        for hc, norm, f in subs:
            y = f(layer_norm(hyper_read(xs, W[p + hc + ".in"]), W[p + norm], eps))
            xs = hyper_write(xs, W[p + hc + ".mix"], W[p + hc + ".out"], y, mult)
        if layers_out is not None:
            layers_out.append(xs.sum(axis=0))
    return soft_cap(layer_norm(xs.sum(axis=0), W["final.norm"], eps) @ W["head"].T, dtype(cfg["logit_softcap"]))


MIXERS = {"delta": gated_delta_mixer, "delta_2": gated_delta_mixer, "latent_attention": latent_attention_mixer}


def forward(cfg, weights, tokens, dtype=np.float64, layers_out=None):
    """Logits [T, vocab] of a "Bofirax" or "Zekilix" configuration; layers_out (a list) receives the residual
    stream (the sum of the streams, if there are several) after every layer."""
    W = {n: np.asarray(a, dtype=dtype) for n, a in weights.items()}
    if cfg["architecture"] == "Zekilix":
        return forward_hyper(cfg, W, tokens, dtype, layers_out)
    eps = dtype(cfg["norm"]["eps"])
    x = W["embed"][np.asarray(tokens, dtype=np.int64)]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}"
        y = MIXERS[layer["type"]](x, W, p + ".mix", layer["mixer"], eps)
        x = x + rms_norm(y, W[p + ".norm1"], eps) * W[p + ".ls1"]
        if layer["mlp"] is not None:
            y = dense_ff(x, W, p + ".mlp")
            x = x + rms_norm(y, W[p + ".norm2"], eps) * W[p + ".ls2"]
        if layers_out is not None:
            layers_out.append(x)
    return rms_norm(x, W["final.norm"], eps) @ W["embed"].T
