"""Plain float64 model of the Defosun design, token by token, one
function per mechanism.  It shares no code with the engine: weights come
in as a dict of numpy arrays under the checkpoint's tensor names, the
configuration as the parsed config.json dict.

Notation: D model width, T tokens of ONE sequence, B residual streams, H
query heads, G key/value heads, N query/key entries per head (of which
the latent form rotates E more), P value entries per head, R latent
width.
"""
from __future__ import annotations

import numpy as np


def rms_unit(x, eps):
    """x scaled to unit root mean square over the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def zero_centred_norm(x, w, eps):
    """RMS norm whose weight is stored around zero."""
    return rms_unit(x, eps) * (1.0 + w)


def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softmax(s):
    p = np.exp(s - s.max())
    return p / p.sum()


def softmax_with_sink(s, sink):
    """Weights of the scores s beside one more exponential that carries
    no value."""
    m = max(float(s.max()), sink)
    p = np.exp(s - m)
    return p / (p.sum() + np.exp(sink - m))


# ---------------------------------------------------------------------------
# residual streams
# ---------------------------------------------------------------------------
def stream_input(X, a):
    """X [B, T, D] -> the sublayer's input sum_b a_b X_b."""
    return np.tensordot(a, X, axes=(0, 0))


def stream_update(X, M, c, y):
    """New X_t = sum_b M[b, t] X_b + c_t y, all from the old streams."""
    return np.stack([sum(M[b, t] * X[b] for b in range(X.shape[0]))
                     + c[t] * y for t in range(X.shape[0])])


# ---------------------------------------------------------------------------
# rotation
# ---------------------------------------------------------------------------
def rotary_frequencies(rot):
    dims, base = rot["dims"], rot["base"]
    return [base ** (-2.0 * i / dims) for i in range(dims // 2)]


def rotate(x, rot, pairs, positions=None):
    """x [T, heads, E]; pairs[i] = the two entries that turn by position *
    frequency_i; entries outside the pairs pass."""
    y = x.copy()
    for t in range(x.shape[0]):
        p = t if positions is None else positions[t]
        for (a, b), f in zip(pairs, rotary_frequencies(rot)):
            c, s = np.cos(p * f), np.sin(p * f)
            u, w = x[t, :, a], x[t, :, b]
            y[t, :, a] = u * c - w * s
            y[t, :, b] = w * c + u * s
    return y


def rotate_halves(x, rot, positions=None):
    h = rot["dims"] // 2
    return rotate(x, rot, [(i, i + h) for i in range(h)], positions)


def rotate_neighbours(x, rot, positions=None):
    h = rot["dims"] // 2
    return rotate(x, rot, [(2 * i, 2 * i + 1) for i in range(h)], positions)


# ---------------------------------------------------------------------------
# attention whose values are its unrotated keys
# ---------------------------------------------------------------------------
def sink_attention(q, k, v, scale, sink, rows=None):
    """q [T, H, N], k [T, G, N], v [T, G, P]; causal, one sink a head.
    rows: only these positions' outputs."""
    T, H = q.shape[:2]
    G = k.shape[1]
    rows = range(T) if rows is None else rows
    out = np.zeros((len(rows), H, v.shape[2]))
    for n, i in enumerate(rows):
        for h in range(H):
            g = h // (H // G)
            w = softmax_with_sink(k[:i + 1, g] @ q[i, h] * scale, sink[h])
            out[n, h] = w @ v[:i + 1, g]
    return out


def attention_mixer(h, W, pre, m):
    H, G, N = m["heads"], m["kv_heads"], m["dim"]
    T = h.shape[0]
    q = (h @ W[pre + "q"].T + W[pre + "q.b"]).reshape(T, H, N)
    k = (h @ W[pre + "k"].T + W[pre + "k.b"]).reshape(T, G, N)
    o = sink_attention(rotate_halves(q, m["rot"]),
                       rotate_halves(k, m["rot"]), k, m["scale"],
                       W[pre + "sink"])
    return o.reshape(T, H * N) @ W[pre + "o"].T + W[pre + "o.b"]


# ---------------------------------------------------------------------------
# latent attention
# ---------------------------------------------------------------------------
def latent_mixer(h, W, pre, m, eps):
    H, N, E, P, R = (m["heads"], m["dim"], m["rot_dim"], m["vdim"],
                     m["kv_rank"])
    T = h.shape[0]
    q = (h @ W[pre + "q"].T).reshape(T, H, N + E)
    d = h @ W[pre + "dkv"].T
    c = rms_unit(d[:, :R], eps) * W[pre + "dkv.norm"]
    kr = rotate_neighbours(d[:, None, R:], m["rot"])
    kn = (c @ W[pre + "uk"].T).reshape(T, H, N)
    v = (c @ W[pre + "uv"].T).reshape(T, H, P)
    q = np.concatenate([q[:, :, :N], rotate_neighbours(q[:, :, N:],
                                                       m["rot"])], -1)
    k = np.concatenate([kn, np.repeat(kr, H, axis=1)], -1)
    o = sink_attention(q, k, v, m["scale"], W[pre + "sink"])
    return o.reshape(T, H * P) @ W[pre + "o"].T


# ---------------------------------------------------------------------------
# linear attention with one fixed decay per head
# ---------------------------------------------------------------------------
def decayed_memory(q, k, v, decay, S=None):
    """q, k [T, H, N], v [T, H, P]; S [H, N, P] at the start (zero when
    not given).  Returns (read-outs [T, H, P], S at the end)."""
    T, H, N = q.shape
    S = np.zeros((H, N, v.shape[2])) if S is None else S.copy()
    out = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        for h in range(H):
            S[h] = decay[h] * S[h] + np.outer(k[t, h], v[t, h])
            out[t, h] = S[h].T @ q[t, h]
    return out, S


def lightning_mixer(h, W, pre, m, eps):
    H, N, P = m["heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = silu(h @ W[pre + "q"].T).reshape(T, H, N)
    k = silu(h @ W[pre + "k"].T).reshape(T, H, N)
    v = silu(h @ W[pre + "v"].T).reshape(T, H, P)
    o, _ = decayed_memory(q, k, v, m["decay"])
    y = rms_unit(o.reshape(T, H * P), eps) * W[pre + "norm"]
    return (y * sigmoid(h @ W[pre + "g"].T)) @ W[pre + "o"].T


# ---------------------------------------------------------------------------
# feed-forwards
# ---------------------------------------------------------------------------
def dense_ff(h, W, pre):
    return (silu(h @ W[pre + "gate"].T) * (h @ W[pre + "up"].T)) \
        @ W[pre + "down"].T


def clamped_expert(h, W, pre, limit):
    g = np.minimum(h @ W[pre + "gate"].T, limit)
    u = np.clip(h @ W[pre + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ W[pre + "down"].T


def route(z, top):
    """[(expert, weight)]: the `top` largest entries of softmax(z), kept
    as they are."""
    s = softmax(z)
    return [(e, s[e]) for e in np.argsort(-s, kind="stable")[:top]]


def moe_ff(h, W, pre, f):
    out = np.zeros((h.shape[0], W[pre + "e0.down"].shape[0]))
    for t, z in enumerate(h @ W[pre + "router"].T):
        for e, w in route(z, f["router"]["top"]):
            out[t] += w * clamped_expert(h[t], W, f"{pre}e{e}.",
                                         f["expert"]["limit"])
    if f.get("shared") is not None:
        y = clamped_expert(h, W, pre + "shared.", f["shared"]["limit"])
        out += sigmoid(h @ W[pre + "shared.sg"].T) * y
    return out


# ---------------------------------------------------------------------------
# the model
# ---------------------------------------------------------------------------
def layer_runs(cfg):
    """Layer numbers in the order they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] \
        + list(range(b, n))


def forward(W, cfg, tokens):
    """Returns (logits [T, vocab], sum of the streams after every layer
    run [runs, T, D])."""
    eps = cfg["norm"]["eps"]
    x = W["embed"][np.asarray(tokens)]
    X = np.stack([x] * cfg["streams"])
    taps = []
    for i in layer_runs(cfg):
        l, p = cfg["layers"][i], f"l{i}."
        h = zero_centred_norm(stream_input(X, W[p + "hc1.in"]),
                              W[p + "norm1"], eps)
        if l["type"] == "attention":
            y = attention_mixer(h, W, p + "mix.", l["mixer"])
        elif l["type"] == "latent_attention":
            y = latent_mixer(h, W, p + "mix.", l["mixer"], eps)
        elif l["type"] == "lightning":
            y = lightning_mixer(h, W, p + "mix.", l["mixer"], eps)
        else:
            raise ValueError(l["type"])
        X = stream_update(X, W[p + "hc1.mix"], W[p + "hc1.out"], y)
        f = l.get("mlp")
        if f is not None:
            h = zero_centred_norm(stream_input(X, W[p + "hc2.in"]),
                                  W[p + "norm2"], eps)
            y = dense_ff(h, W, p + "mlp.") if f["kind"] == "dense" \
                else moe_ff(h, W, p + "mlp.", f)
            X = stream_update(X, W[p + "hc2.mix"], W[p + "hc2.out"], y)
        taps.append(X.sum(0))
    logits = zero_centred_norm(X.sum(0), W["final.norm"], eps) \
        @ W["head"].T
    return logits, np.stack(taps)


# ---------------------------------------------------------------------------
# random checkpoints for the tests
# ---------------------------------------------------------------------------
def tensor_shapes(cfg):
    """Tensor name -> shape of a checkpoint of this configuration."""
    D, V, B = cfg["width"], cfg["vocab"], cfg["streams"]
    sh = {"embed": (V, D), "final.norm": (D,), "head": (V, D)}

    def unit(pre, ff):
        sh.update({pre + "gate": (ff, D), pre + "up": (ff, D),
                   pre + "down": (D, ff)})

    for i, l in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", l["mixer"], l.get("mlp")
        x = p + "mix."
        H, N, P = m["heads"], m["dim"], m["vdim"]
        for q in (1, 2) if f is not None else (1,):
            sh.update({p + f"norm{q}": (D,), p + f"hc{q}.in": (B,),
                       p + f"hc{q}.out": (B,), p + f"hc{q}.mix": (B, B)})
        sh[x + "o"] = (D, H * P)
        if l["type"] == "attention":
            GN = m["kv_heads"] * N
            sh.update({x + "q": (H * N, D), x + "q.b": (H * N,),
                       x + "k": (GN, D), x + "k.b": (GN,),
                       x + "sink": (H,), x + "o.b": (D,)})
        elif l["type"] == "latent_attention":
            E, R = m["rot_dim"], m["kv_rank"]
            sh.update({x + "q": (H * (N + E), D), x + "dkv": (R + E, D),
                       x + "dkv.norm": (R,), x + "uk": (H * N, R),
                       x + "uv": (H * P, R), x + "sink": (H,)})
        else:
            sh.update({x + "q": (H * N, D), x + "k": (H * N, D),
                       x + "v": (H * P, D), x + "g": (H * P, D),
                       x + "norm": (H * P,)})
        if f is None:
            continue
        if f["kind"] == "dense":
            unit(p + "mlp.", f["ff"])
            continue
        E = f["router"]["experts"]
        sh[p + "mlp.router"] = (E, D)
        for e in range(E):
            unit(p + f"mlp.e{e}.", f["expert"]["ff"])
        if f.get("shared") is not None:
            unit(p + "mlp.shared.", f["shared"]["ff"])
            sh[p + "mlp.shared.sg"] = (1, D)
    return sh


def random_weights(cfg, seed=0):
    """Random weights, rounded to bfloat16 (what a checkpoint stores),
    as float64 arrays.  Stream matrices lean towards the identity."""
    import torch

    g = torch.Generator().manual_seed(seed)
    B = cfg["streams"]
    W = {}
    for name, shape in tensor_shapes(cfg).items():
        x = torch.randn(shape, generator=g, dtype=torch.float32)
        last = name.rsplit(".", 1)[-1]
        if name.endswith(".mix") and ".hc" in name:
            x = torch.eye(B) * 0.8 + x * 0.3 / B
        elif ".hc" in name:
            x = (1.0 if last == "out" else 1.0 / B) * (1.0 + 0.3 * x)
        elif last in ("norm1", "norm2") or name == "final.norm":
            x = x * 0.2
        elif last == "norm":
            x = 1.0 + x * 0.2
        elif last == "b":
            x = x * 0.3
        elif last == "router":
            x = x * 2.0 * shape[1] ** -0.5
        elif len(shape) == 2 and name != "embed":
            x = x * 1.2 * shape[1] ** -0.5
        W[name] = x.to(torch.bfloat16).double().numpy()
    return W


def save_checkpoint(path, cfg, W):
    """config.json + model.safetensors (bfloat16) in `path`."""
    import json
    import os

    import torch
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: torch.from_numpy(v).to(torch.bfloat16).contiguous()
               for k, v in W.items()},
              os.path.join(path, "model.safetensors"))
    return str(path)


def make_config(width, vocab, layers, streams=2, loop=None, eps=1e-5):
    """loop: (start, stop, times) or None."""
    c = {"architecture": "Defosun", "width": width, "vocab": vocab,
         "norm": {"eps": eps}, "streams": streams, "layers": layers}
    if loop is not None:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, limit, shared=None):
    """shared: (ff, limit) or None."""
    f = {"kind": "moe", "router": {"experts": experts, "top": top},
         "expert": {"ff": ff, "limit": limit}}
    if shared is not None:
        f["shared"] = {"ff": shared[0], "limit": shared[1]}
    return f


def attention_layer(heads, kv_heads, dim, rot_dims, base, scale, mlp=None):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                      "vdim": dim, "scale": scale,
                      "rot": {"dims": rot_dims, "base": base}}}


def latent_layer(heads, dim, rot_dim, vdim, kv_rank, base, scale, mlp=None):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim,
                      "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
                      "rot": {"dims": rot_dim, "base": base}}}


def lightning_layer(heads, dim, vdim, decay, mlp=None):
    return {"type": "lightning", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim,
                      "decay": list(decay)}}
