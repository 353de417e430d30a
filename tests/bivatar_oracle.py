"""Plain float64 model of the Bivatar design, token by token, one
function per mechanism.  It shares no code with the engine: weights come
in as a dict of numpy arrays under the checkpoint's tensor names, the
configuration as the parsed config.json dict.

Notation: D model width, T tokens of ONE sequence, H query heads, G
key/value heads, N query/key entries per head (of which the latent form
rotates E more), P value entries per head, R latent width.
"""
from __future__ import annotations

import math

import numpy as np


def rms_unit(x, eps):
    """x scaled to unit root mean square over the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi)
                                    * (z + 0.044715 * z ** 3)))


def softmax(s):
    p = np.exp(s - s.max())
    return p / p.sum()


# ---------------------------------------------------------------------------
# windowed attention with kept first tokens and a distance bias
# ---------------------------------------------------------------------------
def distance_slopes(H):
    return [2.0 ** (-8.0 * (h + 1) / H) for h in range(H)]


def visible(i, window, keep):
    """Positions that position i attends to: the last `window` ones and
    the first `keep` of the sequence."""
    return [j for j in range(i + 1)
            if not window or i - j < window or j < keep]


def window_attention(q, k, v, H, G, scale, window, keep, slopes=None,
                     rows=None):
    """q [T, H, N], k [T, G, N], v [T, G, P]; score = q.k * scale -
    slope_h (i - j) over the visible j, softmax.  rows: only these
    positions' outputs."""
    rows = range(q.shape[0]) if rows is None else rows
    slopes = distance_slopes(H) if slopes is None else slopes
    out = np.zeros((len(rows), H, v.shape[2]))
    for n, i in enumerate(rows):
        js = np.array(visible(i, window, keep))
        for h in range(H):
            g = h // (H // G)
            s = k[js, g] @ q[i, h] * scale - slopes[h] * (i - js)
            out[n, h] = softmax(s) @ v[js, g]
    return out


def attention_mixer(h, W, pre, m, eps):
    H, G, N, P = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = (h @ W[pre + "q"].T).reshape(T, H, N)
    k = (h @ W[pre + "k"].T).reshape(T, G, N)
    v = (h @ W[pre + "v"].T).reshape(T, G, P)
    q = rms_unit(q, eps) * W[pre + "q.norm"]
    k = rms_unit(k, eps) * W[pre + "k.norm"]
    mask = m.get("mask") or {}
    o = window_attention(q, k, v, H, G, m["scale"], mask.get("size", 0),
                         mask.get("keep_first", 0))
    o = o * sigmoid(h @ W[pre + "g"].T)[:, :, None]
    return o.reshape(T, H * P) @ W[pre + "o"].T


# ---------------------------------------------------------------------------
# latent attention
# ---------------------------------------------------------------------------
def rotary_frequencies(rot):
    """Angular step per rotated pair, and the factor on cos and sin."""
    dims, base = rot["dims"], rot["base"]
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return np.array(f), 1.0

    def where(turns):
        return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) \
            / (2.0 * math.log(base))

    lo = max(math.floor(where(sc["fast"])), 0)
    hi = min(math.ceil(where(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * ramp + fi * (1.0 - ramp))
    return np.array(out), 0.1 * math.log(sc["factor"]) + 1.0


def rotate_halves(x, rot, positions=None):
    """x [T, heads, E]: entry i is paired with entry i + dims/2 and the
    pair turned by position * frequency_i; entries past dims pass."""
    freq, mag = rotary_frequencies(rot)
    half = rot["dims"] // 2
    y = x.copy()
    for t in range(x.shape[0]):
        p = t if positions is None else positions[t]
        for i, f in enumerate(freq):
            c, s = math.cos(p * f) * mag, math.sin(p * f) * mag
            u, w = x[t, :, i], x[t, :, i + half]
            y[t, :, i] = u * c - w * s
            y[t, :, i + half] = w * c + u * s
    return y


def latent_keys(h, W, pre, m, eps):
    """(latent [T, R], rotated shared key [T, E]): what a token leaves
    for the tokens after it."""
    R = m["kv_rank"]
    d = h @ W[pre + "dkv"].T
    c = rms_unit(d[:, :R], eps) * W[pre + "dkv.norm"]
    return c, rotate_halves(d[:, None, R:], m["rot"])[:, 0]


def latent_attention(q, kn, kr, v, N, scale):
    """q [T, H, N + E] with the last E entries rotated, kn [T, H, N]
    per-head keys, kr [T, E] the shared rotated key, v [T, H, P];
    causal."""
    T, H = q.shape[:2]
    out = np.zeros((T, H, v.shape[2]))
    for i in range(T):
        for h in range(H):
            s = (kn[:i + 1, h] @ q[i, h, :N]
                 + kr[:i + 1] @ q[i, h, N:]) * scale
            out[i, h] = softmax(s) @ v[:i + 1, h]
    return out


def latent_mixer(h, W, pre, m, eps, kv=None):
    """Returns (output, (latent, rotated key)); `kv` given = another
    layer's."""
    H, N, E, P = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    T = h.shape[0]
    cq = rms_unit(h @ W[pre + "dq"].T, eps) * W[pre + "dq.norm"]
    q = (cq @ W[pre + "uq"].T).reshape(T, H, N + E)
    q = np.concatenate([q[:, :, :N], rotate_halves(q[:, :, N:], m["rot"])],
                       -1)
    if kv is None:
        kv = latent_keys(h, W, pre, m, eps)
    c, kr = kv
    kn = (c @ W[pre + "uk"].T).reshape(T, H, N)
    v = (c @ W[pre + "uv"].T).reshape(T, H, P)
    o = latent_attention(q, kn, kr, v, N, m["scale"])
    o = o * sigmoid(h @ W[pre + "g"].T)[:, :, None]
    return o.reshape(T, H * P) @ W[pre + "o"].T, kv


def gated_ff(h, W, pre):
    return (gelu_tanh(h @ W[pre + "gate"].T) * (h @ W[pre + "up"].T)) \
        @ W[pre + "down"].T


def forward(W, cfg, tokens):
    """Returns (logits [T, vocab], residual after every layer
    [layers, T, D])."""
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    tokens = np.asarray(tokens)
    x = W["embed"][tokens] * cfg["embedding"]["scale"]
    kv_of, taps = {}, []
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        if l["type"] == "attention":
            d = attention_mixer(x, W, p + "mix.", m, eps)
        elif l["type"] == "latent_attention":
            src = m.get("kv_from")
            d, kv_of[i] = latent_mixer(x, W, p + "mix.", m, eps,
                                       None if src is None else kv_of[src])
        else:
            raise ValueError(l["type"])
        x = x + mult * rms_unit(d, eps) * W[p + "norm1"]
        if l.get("mlp") is not None:
            d = gated_ff(x, W, p + "mlp.")
            x = x + mult * rms_unit(d, eps) * W[p + "norm2"]
        taps.append(x.copy())
    logits = (rms_unit(x, eps) * W["final.norm"]) @ W["head"].T
    return logits, np.stack(taps)


# ---------------------------------------------------------------------------
# random checkpoints for the tests
# ---------------------------------------------------------------------------
def tensor_shapes(cfg):
    """Tensor name -> shape of a checkpoint of this configuration."""
    D, V = cfg["width"], cfg["vocab"]
    sh = {"embed": (V, D), "final.norm": (D,), "head": (V, D)}
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        q = p + "mix."
        H, N, P = m["heads"], m["dim"], m["vdim"]
        sh.update({p + "norm1": (D,), q + "g": (H, D), q + "o": (D, H * P)})
        if l["type"] == "attention":
            G = m["kv_heads"]
            sh.update({q + "q": (H * N, D), q + "k": (G * N, D),
                       q + "v": (G * P, D), q + "q.norm": (N,),
                       q + "k.norm": (N,)})
        else:
            E, R, Q = m["rot_dim"], m["kv_rank"], m["q_rank"]
            sh.update({q + "dq": (Q, D), q + "dq.norm": (Q,),
                       q + "uq": (H * (N + E), Q), q + "uk": (H * N, R),
                       q + "uv": (H * P, R)})
            if m.get("kv_from") is None:
                sh.update({q + "dkv": (R + E, D), q + "dkv.norm": (R,)})
        f = l.get("mlp")
        if f is not None:
            ff = f["ff"]
            sh.update({p + "norm2": (D,), p + "mlp.gate": (ff, D),
                       p + "mlp.up": (ff, D), p + "mlp.down": (D, ff)})
    return sh


def random_weights(cfg, seed=0):
    """Random weights, rounded to bfloat16 (what a checkpoint stores),
    as float64 arrays."""
    import torch

    g = torch.Generator().manual_seed(seed)
    W = {}
    for name, shape in tensor_shapes(cfg).items():
        x = torch.randn(shape, generator=g, dtype=torch.float32)
        last = name.rsplit(".", 1)[-1]
        if name == "embed":
            x = x / cfg["embedding"]["scale"]
        elif last in ("norm1", "norm2", "norm"):
            x = 1.0 + x * 0.2
        elif len(shape) == 2:
            x = x * shape[1] ** -0.5 * (3.0 if last == "g" else 1.5)
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


def make_config(width, vocab, layers, scale=None, mult=0.5, eps=1e-5):
    return {"architecture": "Bivatar", "width": width, "vocab": vocab,
            "norm": {"eps": eps}, "residual_mult": mult,
            "embedding": {"scale": scale or float(width) ** 0.5},
            "layers": layers}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def attention_layer(heads, kv_heads, dim, vdim, window, keep, scale,
                    mlp=None):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                      "vdim": vdim, "scale": scale,
                      "mask": {"size": window, "keep_first": keep}}}


def rot(dims, base=10000.0, factor=None, original=None, fast=32.0,
        slow=1.0):
    r = {"dims": dims, "base": base}
    if factor:
        r["scaling"] = {"factor": factor, "original": original,
                        "fast": fast, "slow": slow}
    return r


def latent_layer(heads, dim, rotary, vdim, kv_rank, q_rank, scale, mlp=None,
                 kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rotary["dims"],
         "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
         "scale": scale, "rot": rotary}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}
