#!/usr/bin/env python3
"""Defosun beside Bozolorn at equal layer sizes: engine prefill / decode
throughput and per-kernel roofline fractions (random weights).

Run through `python bench.py --arch-compare --arch defosun [--arch-size
NAME]`; prints one JSON object.  Bozolorn is the closest model the engine
serves: rotated softmax attention with a sink, a recurrent outer-product
memory, clamped experts, an fp32 residual, eager decode.  Both models get
4 layers of the same width, head counts and head sizes, and the same
routed experts in every layer; Defosun has four residual streams, latent
attention in one layer and a shared expert on top.  Same two measurements
as tools/bench_hybrid.py: the LLMEngine loop for both models, and each
kernel in the form this design launches next to the like kernel of
Bozolorn, Bivatar or Feditar, priced against the MI355X roofline (2.5
PFLOP/s dense bf16, 8 TB/s HBM).
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
    "4k": dict(width=4096, heads=32, kv_heads=8, dim=128, rot_dims=64,
               kv_rank=512, rot_dim=64, ff=14336, experts=8, top=2,
               streams=4, chunk=1024, vocab=32000),
    "2k": dict(width=2048, heads=16, kv_heads=4, dim=128, rot_dims=64,
               kv_rank=256, rot_dim=64, ff=8192, experts=8, top=2,
               streams=4, chunk=1024, vocab=32000),
}


def _configs(sz):
    from inference_gateway_amd.engine.config import (bozolorn_preset,
                                                     defosun_preset)

    dfo = defosun_preset(
        "defosun-bench", width=sz["width"], vocab=sz["vocab"],
        pattern="am fm am lm", heads=sz["heads"], kv_heads=sz["kv_heads"],
        dim=sz["dim"], rot_dims=sz["rot_dims"], l_dim=sz["dim"],
        rot_dim=sz["rot_dim"], l_vdim=sz["dim"], kv_rank=sz["kv_rank"],
        d_dim=sz["dim"], d_vdim=sz["dim"], ff=sz["ff"],
        experts=sz["experts"], top=sz["top"],
        expert_ff=sz["ff"] // sz["top"], shared_ff=sz["ff"] // 4,
        streams=sz["streams"])
    boz = bozolorn_preset(
        "bozolorn-bench", width=sz["width"], vocab=sz["vocab"],
        pattern="pm am pm a1m", heads=sz["heads"], kv_heads=sz["kv_heads"],
        dim=sz["dim"], vdim=sz["dim"], chunk=sz["chunk"],
        rot_dims=sz["rot_dims"], d_heads=sz["heads"],
        d_kv_heads=sz["kv_heads"], d_dim=sz["dim"], d_vdim=sz["dim"],
        experts=sz["experts"], top=sz["top"], groups=4, keep=2,
        expert_ff=sz["ff"] // sz["top"], side_dim=64, yarn_factor=4.0,
        yarn_original=4096.0)
    return dfo, boz


def _kernels(sz):
    from inference_gateway_amd import ops

    dev, bf = "cuda", torch.bfloat16
    D, H, G, N, R, RD = (sz[k] for k in ("width", "heads", "kv_heads",
                                         "dim", "kv_rank", "rot_dim"))
    P = N
    out = {}
    bs = 16

    def table(nseq, ctx):
        return (torch.arange(nseq * (ctx // bs), dtype=torch.int32,
                             device=dev) + 1).view(nseq, ctx // bs)

    def seqs(nseq, L, start):
        T = nseq * L
        cu = torch.arange(0, T + 1, L, dtype=torch.int32, device=dev)
        st = torch.full((nseq,), start, dtype=torch.int32, device=dev)
        sl = torch.arange(nseq, dtype=torch.int32, device=dev)
        return T, cu, st, sl, sl.repeat_interleave(L)

    learned = torch.randn(H, device=dev)
    zero = torch.zeros(H, device=dev)

    # ---- attention: 4 x 2048 prompt rows; 256 decoded rows at 2048 ----
    for tag, nseq, L, ctx, it in (("prompt", 4, 2048, 2048, 4),
                                  ("decode", 256, 1, 2048, 10)):
        T, cu, st, _sl, row_seq = seqs(nseq, L, ctx - L)
        pos = torch.arange(ctx - L, ctx, dtype=torch.int32,
                           device=dev).repeat(nseq)
        bt = table(nseq, ctx)
        nb = nseq * (ctx // bs) + 1
        keys = nseq * sum(range(ctx - L + 1, ctx + 1))
        pre = T if L > 1 else 0
        lens = [L] * nseq if L > 1 else None
        kc = torch.randn(nb, G, bs, N, device=dev, dtype=bf)
        vc = torch.randn(nb, G, bs, P, device=dev, dtype=bf)
        q = torch.randn(T, H * N, device=dev, dtype=bf)
        mem = 2.0 * G * (N + P) if L == 1 else 0.0
        for name, s in (("tied_attention", learned),
                        ("sink_attention", zero)):
            t = _time(lambda: ops.softcap_attention(
                q, kc, vc, bt, row_seq, pos, 0.09, 0.0, 0.0, 1, 0, pre,
                lens, cu, st, sinks=s), it)
            out[f"{name}_{tag}"] = _entry(
                t, flops=2.0 * keys * H * (N + P), bytes_=keys * mem)
        del kc, vc
        # the query as this design hands it over: the rotated part is a
        # slice of the fused projection's row
        W = H * (N + RD) + R + RD
        proj = torch.randn(T, W, device=dev, dtype=bf)
        qr = proj[:, :H * (N + RD)].view(T, H, N + RD)[:, :, N:]
        qr2 = torch.randn(T, H, N + RD, device=dev, dtype=bf)[:, :, N:]
        qa = torch.randn(H, T, R, device=dev, dtype=bf).transpose(0, 1)
        cache = torch.randn(nb, bs, R + RD, device=dev, dtype=bf)
        gate = torch.rand(T, H, device=dev)
        mem = 2.0 * (R + RD) if L == 1 else 0.0
        for name, x, s, g in (("latent_direct", qr, learned, None),
                              ("latent_gated", qr2, None, gate)):
            t = _time(lambda: ops.latent_attention(
                qa, x, cache, bt, row_seq, pos, s, 0.05, 0, pre, lens, ctx,
                gate=g), it)
            out[f"{name}_{tag}"] = _entry(
                t, flops=2.0 * keys * H * (2 * R + RD), bytes_=keys * mem)
        del cache, proj, qa, qr2

    # ---- memory scans ----
    for tag, nseq, L, start in (("prompt", 64, 1024, 0),
                                ("one_prompt", 1, 8192, 0),
                                ("decode", 256, 1, 5)):
        T, cu, st, sl, _rs = seqs(nseq, L, start)
        it = 5 if L > 1 else 20
        proj = torch.randn(T, 2 * H * (N + P), device=dev, dtype=bf)
        k0, v0, g0 = H * N, 2 * H * N, 2 * H * N + H * P
        q, k, v = (proj[:, :k0].view(T, H, N), proj[:, k0:v0].view(T, H, N),
                   proj[:, v0:g0].view(T, H, P))
        decay = torch.linspace(0.5, 0.999, H, device=dev)
        mem = torch.zeros(nseq, H * N * P, device=dev)
        io = T * H * (2 * N + P) * 2.0 + T * H * P * 4.0 \
            + (2.0 if start else 1.0) * mem.numel() * 4
        fl = 4.0 * T * H * N * P
        t = _time(lambda: ops.fixed_decay_scan(q, k, v, decay, mem, cu, st,
                                               sl, [L] * nseq), it)
        out[f"fixed_decay_{tag}"] = _entry(t, flops=fl, bytes_=io)
        # the like kernel: Feditar's scalar-decay outer-product memory
        a3 = decay.expand(T, H).unsqueeze(-1).contiguous()
        t = _time(lambda: ops.outer_scan(
            q, k, v, a3, None, None, None, mem, cu, st, sl, [L] * nseq,
            ops.DECAY_LINEAR, False, 1.0), min(it, 5))
        out[f"outer_scan_{tag}"] = _entry(t, flops=fl, bytes_=io)
        o = torch.randn(T, H, P, device=dev)
        w = torch.ones(H * P, device=dev)
        for name, group, act in (("head_norm_gate_all", H * P,
                                  ops.GATE_SIGMOID),
                                 ("head_norm_gate_each", P, ops.GATE_SILU)):
            t = _time(lambda: ops.head_norm_gate(
                o, proj[:, g0:], w, 1e-6, group, act, False, None, None,
                bf), it)
            out[f"{name}_{tag}"] = _entry(t, bytes_=T * H * P * 8.0)
        del proj, q, k, v, mem, a3, o

    # ---- row kernels on 8192 rows (8 sequences of 1024) ----
    T = 8192
    B = sz["streams"]
    pos = torch.arange(1024, dtype=torch.int32, device=dev).repeat(8)
    slots = torch.arange(bs, T + bs, dtype=torch.int32, device=dev)
    dl = torch.randn(T, D, device=dev, dtype=bf)
    w = torch.ones(D, device=dev)
    for rows in (T, 64):
        st = torch.randn(rows, B, D, device=dev)
        mix = torch.eye(B, device=dev)
        one = torch.full((B,), 1e-3, device=dev)
        t = _time(lambda: ops.stream_step(st, dl[:rows], mix, one, one, w,
                                          1e-5, bf))
        out[f"stream_step_{rows}"] = _entry(
            t, bytes_=rows * D * (8.0 * B + 4))
        res = torch.randn(rows, D, device=dev)
        t = _time(lambda: ops.add_normed_rmsnorm(res, dl[:rows], w, w, 1e-5,
                                                 bf))
        out[f"add_normed_rmsnorm_{rows}"] = _entry(t, bytes_=rows * D * 12.0)
    inv = torch.rand(sz["rot_dims"] // 2, device=dev)
    wn = torch.ones(N, device=dev)
    kcs = torch.zeros(T // bs + 1, G, bs, N, device=dev, dtype=bf)
    vcs = torch.zeros(T // bs + 1, G, bs, P, device=dev, dtype=bf)
    C = (H + G) * N
    proj = torch.randn(T, C + G * P, device=dev, dtype=bf)
    pt = proj[:, :C].contiguous()
    t = _time(lambda: ops.qk_norm_rope_append(
        pt, pos, slots, kcs, vcs, None, None, inv, 1.0, 1e-5, H, G, N, P,
        half=True, tied=True))
    out["rope_append_tied"] = _entry(t, bytes_=T * (C * 4.0 + G * N * 2.0))
    t = _time(lambda: ops.qk_norm_rope_append(
        proj, pos, slots, kcs, vcs, wn, wn, inv, 1.1, 1e-5, H, G, N, P))
    out["qk_norm_rope_append"] = _entry(t, bytes_=T * (C + G * P) * 4.0)
    inv = torch.rand(RD // 2, device=dev)
    wk = torch.ones(R, device=dev)
    x = torch.randn(T, H * (N + RD) + R + RD, device=dev, dtype=bf)
    lat = torch.zeros(T // bs + 1, bs, R + RD, device=dev, dtype=bf)
    t = _time(lambda: ops.latent_rope_append(x, pos, slots, lat, wk, inv,
                                             1e-5, H, N, RD, R))
    out["latent_rope_append"] = _entry(
        t, bytes_=T * (R + RD + H * RD) * 4.0)
    # the like pair of launches: Fedatar's down-projection step + rotation
    down = torch.randn(T, H + R + RD + H, device=dev, dtype=bf)
    wq = torch.ones(H, device=dev)
    qh = torch.randn(T, H, N + RD, device=dev, dtype=bf)

    def pair():
        ops.latent_down_post(down, pos, slots, lat, wq, wk, inv, 1e-5, H, R,
                             RD, H)
        ops.rope_pairs_(qh, pos, inv, N)

    out["latent_down_post+rope_pairs"] = _entry(
        _time(pair), bytes_=T * (R + RD + H * RD) * 4.0)

    # ---- experts: activation, router, dispatch ----
    K, E, F_ = sz["top"], sz["experts"], sz["ff"] // sz["top"]
    gu = torch.randn(T * K, 2 * F_, device=dev, dtype=bf)
    for name, args in (("gated_act_clamped", (ops.GATED_ACT_CLAMPED, 7.0,
                                              1.702)),
                       ("gated_act_silu", (ops.GATED_ACT_SILU,))):
        t = _time(lambda: ops.gated_act(gu, *args))
        out[name] = _entry(t, bytes_=T * K * F_ * 6.0)
    del gu
    for rows in (256, T):
        lg = torch.randn(rows, E + 1, device=dev)
        lc = lg[:, :E].contiguous()
        cap = rows if rows <= 256 else 0
        for name, z, all_ in (("softmax_route", lg[:, :E], True),
                              ("moe_topk_route", lc, False)):
            t = _time(lambda: ops.moe_topk_route(z, K, cap, over_all=all_))
            out[f"{name}_{rows}"] = _entry(t, bytes_=rows * (E * 4.0
                                                             + K * 16.0))
    wt = torch.rand(T, K, device=dev)
    dst = torch.randperm(T * K, device=dev)
    y = torch.randn(T * K, D, device=dev, dtype=bf)
    sg = torch.randn(T, device=dev)
    t = _time(lambda: ops.moe_combine(y, dst, wt, dl, sg))
    out["moe_combine"] = _entry(t, bytes_=T * D * (K + 2) * 2.0)
    t = _time(lambda: ops.moe_scatter_rows(dl, dst, T * K))
    out["moe_scatter_rows"] = _entry(t, bytes_=T * D * (K + 1) * 2.0)
    return out


def run(size: str = "2k", batch: int = 64, prompt_len: int = 1024,
        steps: int = 32, warmup: int = 4) -> dict:
    sz = SIZES[size]
    dfo, boz = _configs(sz)
    res = {"size": size, "shape": sz, "batch": batch,
           "prompt_len": prompt_len, "steps": steps, "dtype": "bf16",
           "data": "synthetic (random weights and tokens)"}
    res["kernels"] = _kernels(sz)
    res["defosun"] = _engine_run(dfo, batch, prompt_len, steps, warmup)
    res["bozolorn"] = _engine_run(boz, batch, prompt_len, steps, warmup)
    return res


if __name__ == "__main__":
    print(json.dumps(run(*(sys.argv[1:2] or ["2k"]))))
