#!/usr/bin/env python3
"""Bivatar beside Fedatar at equal layer sizes: engine prefill / decode
throughput and per-kernel roofline fractions (random weights).

Run through `python bench.py --arch-compare --arch bivatar [--arch-size
NAME]`; prints one JSON object.  Fedatar is the closest model the engine
serves: latent attention beside dense feed-forwards on an fp32 residual
stream, eager decode.  Both models get 4 layers of the same width, head
counts, head and latent sizes; Bivatar's gated feed-forward (three
matrices) is sized to Fedatar's two-matrix one.  Same two measurements as
tools/bench_hybrid.py: the LLMEngine loop for both models, and each kernel
in the form this design launches next to the like kernel of Fedatar or
Bozolorn, priced against the MI355X roofline (2.5 PFLOP/s dense bf16, 8
TB/s HBM).
"""
from __future__ import annotations

import json
import sys
from pathlib import Path

import torch

sys.path.insert(0, str(Path(__file__).resolve().parent.parent))
sys.path.insert(0, str(Path(__file__).resolve().parent))

from bench_hybrid import _engine_run, _entry, _time  # noqa: E402

# Llama-3-8B's layer shape, and a half-width one
SIZES = {
    "4k": dict(width=4096, heads=32, kv_heads=8, dim=128, vdim=128,
               window=512, keep=16, rot_dim=64, kv_rank=512, q_rank=1536,
               ff=14336, vocab=32000),
    "2k": dict(width=2048, heads=16, kv_heads=4, dim=128, vdim=128,
               window=512, keep=16, rot_dim=64, kv_rank=256, q_rank=768,
               ff=8192, vocab=32000),
}


def _configs(sz):
    from inference_gateway_amd.engine.config import (bivatar_preset,
                                                     fedatar_preset)

    biv = bivatar_preset(
        "bivatar-bench", width=sz["width"], vocab=sz["vocab"],
        pattern="wd ld wd l1d", heads=sz["heads"], kv_heads=sz["kv_heads"],
        dim=sz["dim"], vdim=sz["vdim"], window=sz["window"],
        keep_first=sz["keep"], l_dim=sz["dim"], rot_dim=sz["rot_dim"],
        l_vdim=sz["vdim"], kv_rank=sz["kv_rank"], q_rank=sz["q_rank"],
        ff=sz["ff"], yarn_factor=8.0, yarn_original=4096.0)
    fed = fedatar_preset(
        "fedatar-bench", width=sz["width"], vocab=sz["vocab"],
        pattern="ad ad ad ad", heads=sz["heads"], dim=sz["dim"],
        rot_dim=sz["rot_dim"], vdim=sz["vdim"], kv_rank=sz["kv_rank"],
        q_rank=sz["q_rank"], window=0, ff=sz["ff"] * 3 // 2, experts=1,
        top=1, expert_ff=1, shared_ff=0)
    return biv, fed


def _kernels(sz):
    from inference_gateway_amd import ops

    dev, bf = "cuda", torch.bfloat16
    D, H, G = sz["width"], sz["heads"], sz["kv_heads"]
    N, P, R, RD, QR = (sz[k] for k in ("dim", "vdim", "kv_rank", "rot_dim",
                                       "q_rank"))
    W, keep = sz["window"], sz["keep"]
    out = {}
    bs = 16

    def table(nseq, ctx):
        return (torch.arange(nseq * (ctx // bs), dtype=torch.int32,
                             device=dev) + 1).view(nseq, ctx // bs)

    def paged(nseq, ctx):
        nb = nseq * (ctx // bs) + 1
        return (torch.randn(nb, G, bs, N, device=dev, dtype=bf),
                torch.randn(nb, G, bs, P, device=dev, dtype=bf))

    slopes = torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)],
                          device=dev)
    sink = torch.zeros(H, device=dev)

    def window_pair(tag, n, pos, args, tail, it):
        """Window + kept tokens + per-head gate, and Bozolorn's chunked
        form with its per-entry gate, each on its visible keys."""
        gate1 = torch.randn(n, H, device=dev, dtype=bf)
        gate2 = torch.randn(n, H * P, device=dev, dtype=bf)
        lo = [max(0, p - W + 1) for p in pos]
        keys = sum(p - a + 1 + min(keep, a) for p, a in zip(pos, lo))
        ckeys = sum(p % W + 1 for p in pos)
        mem = 2.0 * G * (N + P) if tag == "decode" else 0.0
        t = _time(lambda: ops.softcap_attention(
            *args, 0.0, 0.0, 1, W, *tail, slopes=slopes, gate=gate1,
            keep=keep), it)
        out[f"window_attention_{tag}"] = _entry(
            t, flops=2.0 * keys * H * (N + P), bytes_=keys * mem)
        t = _time(lambda: ops.softcap_attention(
            *args, 0.0, 0.0, 1, 0, *tail, slopes=slopes, gate=gate2,
            chunk=W), it)
        out[f"chunk_bias_attention_{tag}"] = _entry(
            t, flops=2.0 * ckeys * H * (N + P), bytes_=ckeys * mem)

    # ---- attention: 4 x 2048 prompt rows; 256 decoded rows at 2048 ----
    nseq, L = 4, 2048
    T = nseq * L
    cu = torch.arange(0, T + 1, L, dtype=torch.int32, device=dev)
    st = torch.zeros(nseq, dtype=torch.int32, device=dev)
    row_seq = torch.arange(nseq, dtype=torch.int32,
                           device=dev).repeat_interleave(L)
    pos = torch.arange(L, dtype=torch.int32, device=dev).repeat(nseq)
    bt = table(nseq, L)
    kc, vc = paged(nseq, L)
    q = torch.randn(T, H * N, device=dev, dtype=bf)
    window_pair("prompt", T, list(range(L)) * nseq,
                (q, kc, vc, bt, row_seq, pos, 0.09),
                (T, [L] * nseq, cu, st), 5)

    def latent_pair(tag, rows, keys, args, tail, it, mem=0.0):
        """No sink and the gate fused in, against Fedatar's sink form
        with the same gate."""
        gate = torch.rand(rows, H, device=dev)
        for name, s in (("latent_attention", None),
                        ("latent_sink_attention", sink)):
            t = _time(lambda: ops.latent_attention(
                *args, s, 0.05, 0, *tail, gate=gate), it)
            out[f"{name}_{tag}"] = _entry(
                t, flops=2.0 * keys * H * (2 * R + RD), bytes_=keys * mem)

    cache = torch.randn(nseq * (L // bs) + 1, bs, R + RD, device=dev,
                        dtype=bf)
    qa = torch.randn(T, H, R, device=dev, dtype=bf)
    qr = torch.randn(T, H, RD, device=dev, dtype=bf)
    latent_pair("prompt", T, nseq * L * (L + 1) // 2,
                (qa, qr, cache, bt, row_seq, pos),
                (T, [L] * nseq, L), 3)
    B, ctx = 256, 2048
    bt = table(B, ctx)
    kc, vc = paged(B, ctx)
    rs1 = torch.arange(B, dtype=torch.int32, device=dev)
    pos = torch.full((B,), ctx - 1, dtype=torch.int32, device=dev)
    cu1 = torch.arange(B + 1, dtype=torch.int32, device=dev)
    q = torch.randn(B, H * N, device=dev, dtype=bf)
    window_pair("decode", B, [ctx - 1] * B,
                (q, kc, vc, bt, rs1, pos, 0.09), (0, None, cu1, pos), 10)
    del kc, vc
    cache = torch.randn(B * (ctx // bs) + 1, bs, R + RD, device=dev,
                        dtype=bf)
    latent_pair("decode", B, B * ctx,
                (qa[:B], qr[:B], cache, bt, rs1, pos), (0, None, ctx), 10,
                2.0 * (R + RD))

    # ---- row kernels on 8192 rows (8 sequences of 1024) ----
    T = 8192
    pos = torch.arange(1024, dtype=torch.int32, device=dev).repeat(8)
    slots = torch.arange(bs, T + bs, dtype=torch.int32, device=dev)
    res = torch.randn(T, D, device=dev)
    dl = torch.randn(T, D, device=dev, dtype=bf)
    w = torch.ones(D, device=dev)
    t = _time(lambda: ops.add_normed_rmsnorm(res, dl, w, None, 1e-5, bf,
                                             0.3))
    out["post_norm_add"] = _entry(t, bytes_=T * D * (4 + 4 + 2 + 2.0))
    t = _time(lambda: ops.add_normed_rmsnorm(res, dl, w, w, 1e-5, bf))
    out["add_normed_rmsnorm"] = _entry(t, bytes_=T * D * (4 + 4 + 2 + 2.0))
    t = _time(lambda: ops.add_layernorm(res, dl, w, w, 1e-5, bf))
    out["add_layernorm"] = _entry(t, bytes_=T * D * (4 + 4 + 2 + 2.0))
    C = H * N + G * (N + P)
    proj = torch.randn(T, C + H, device=dev, dtype=bf)
    kcs = torch.zeros(T // bs + 1, G, bs, N, device=dev, dtype=bf)
    vcs = torch.zeros(T // bs + 1, G, bs, P, device=dev, dtype=bf)
    wn = torch.ones(N, device=dev)
    inv = torch.rand(RD // 2, device=dev)
    for name, f in (("qk_norm_append", None), ("qk_norm_rope_append", inv)):
        t = _time(lambda: ops.qk_norm_rope_append(
            proj, pos, slots, kcs, vcs, wn, wn, f, 1.1, 1e-5, H, G, N, P))
        out[name] = _entry(t, bytes_=T * C * 4.0)
    down = torch.randn(T, QR + R + RD + H, device=dev, dtype=bf)
    lat = torch.zeros(T // bs + 1, bs, R + RD, device=dev, dtype=bf)
    wq, wk = torch.ones(QR, device=dev), torch.ones(R, device=dev)
    for name, half in (("latent_down_post_half", True),
                       ("latent_down_post_pairs", False)):
        t = _time(lambda: ops.latent_down_post(
            down, pos, slots, lat, wq, wk, inv, 1e-5, QR, R, RD, H, half,
            1.1))
        out[name] = _entry(t, bytes_=T * (QR + R + RD) * 4.0 + T * H * 6.0)
    qh = torch.randn(T, H, N + RD, device=dev, dtype=bf)
    for name, half in (("rope_half", True), ("rope_pairs", False)):
        t = _time(lambda: ops.rope_pairs_(qh, pos, inv, N, half, 1.1))
        out[name] = _entry(t, bytes_=T * H * RD * 4.0)
    F_ = sz["ff"]
    gu = torch.randn(T, 2 * F_, device=dev, dtype=bf)
    for name, mode in (("gated_act_gelu", ops.GATED_ACT_GELU),
                       ("gated_act_silu", ops.GATED_ACT_SILU)):
        t = _time(lambda: ops.gated_act(gu, mode))
        out[name] = _entry(t, bytes_=T * F_ * 6.0)
    return out


def run(size: str = "2k", batch: int = 64, prompt_len: int = 1024,
        steps: int = 32, warmup: int = 4) -> dict:
    sz = SIZES[size]
    biv, fed = _configs(sz)
    res = {"size": size, "shape": sz, "batch": batch,
           "prompt_len": prompt_len, "steps": steps, "dtype": "bf16",
           "data": "synthetic (random weights and tokens)"}
    res["kernels"] = _kernels(sz)
    res["bivatar"] = _engine_run(biv, batch, prompt_len, steps, warmup)
    res["fedatar"] = _engine_run(fed, batch, prompt_len, steps, warmup)
    return res


if __name__ == "__main__":
    print(json.dumps(run(*(sys.argv[1:2] or ["2k"]))))
