"""Defosun (several residual streams, a repeated run of layers; attention
whose values are its unrotated keys / direct-query latent attention / fixed
decay linear attention; dense and mixture-of-experts feed-forwards)
against a plain float64 model written from the equations
(tests/defosun_oracle.py).

Every test builds its own small configuration and random checkpoint; the
engine reads it through the product loader.  Device-parametrized: the CPU
cases run the reference ops, the GPU cases the HIP kernels, both through
the same engine, cache manager and scheduler.
"""
import json
import os
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import defosun_oracle as oracle
from inference_gateway_amd import ops
from inference_gateway_amd.engine.config import (DefosunConfig,
                                                 EngineConfig,
                                                 SamplingParams)
from inference_gateway_amd.engine.engine import LLMEngine
from inference_gateway_amd.engine.models import moe_common
from inference_gateway_amd.engine.models.registry import (
    is_recurrent, model_config_from_dir)

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]


def _dev(device):
    return "cuda:0" if device == "cuda" else device


def i32(x, device):
    return torch.tensor(x, dtype=torch.int32, device=_dev(device))


def f32(x, device):
    return torch.tensor(np.asarray(x), dtype=torch.float32,
                        device=_dev(device))


def f64(x):
    return x.detach().cpu().double().numpy()


# configurations; sizes all differ from one another
def cfg_small():
    """All mixers and feed-forwards; a loop over the middle."""
    return oracle.make_config(40, 61, [
        oracle.latent_layer(3, 5, 4, 7, 12, 60.0, 0.35,
                            mlp=oracle.moe(5, 3, 14, 1.1, (9, 0.6))),
        oracle.attention_layer(4, 2, 10, 6, 300.0, 0.3,
                               mlp=oracle.dense(18)),
        oracle.lightning_layer(5, 6, 9, [0.3, 0.8, 0.97, 1.0, 0.55],
                               mlp=oracle.moe(4, 1, 11, 0.8)),
        oracle.attention_layer(3, 3, 8, 8, 40.0, 0.4)],
        streams=3, loop=(1, 3, 3))


def cfg_ones():
    """One stream, single heads and groups, one-entry latents and
    memories, one expert, no loop, layers without feed-forward."""
    return oracle.make_config(24, 37, [
        oracle.lightning_layer(1, 1, 1, [0.9]),
        oracle.attention_layer(1, 1, 2, 2, 10.0, 0.6,
                               mlp=oracle.moe(1, 1, 1, 0.5, (1, 2.0))),
        oracle.latent_layer(1, 1, 2, 1, 1, 10.0, 0.6,
                            mlp=oracle.dense(1)),
        oracle.lightning_layer(2, 3, 5, [1.0, 0.0])],
        streams=1, eps=1e-6)


def cfg_wide():
    """Sizes that straddle the kernels' tiles; more streams than the
    in-place step takes; the loop covers every layer."""
    return oracle.make_config(72, 83, [
        oracle.lightning_layer(3, 33, 70, [0.999, 0.7, 0.9],
                               mlp=oracle.dense(50)),
        oracle.latent_layer(5, 33, 20, 70, 68, 1000.0, 0.15,
                            mlp=oracle.moe(9, 4, 17, 1.5, (30, 2.5))),
        oracle.attention_layer(6, 1, 66, 20, 1000.0, 0.12)],
        streams=9, loop=(0, 3, 2))


def cfg_tail():
    """The loop ends with the last layer and starts behind the first;
    odd width; the same layer kind twice in a row inside it."""
    return oracle.make_config(31, 53, [
        oracle.attention_layer(2, 1, 7, 4, 20.0, 0.4,
                               mlp=oracle.dense(13)),
        oracle.lightning_layer(2, 5, 4, [0.95, 0.6]),
        oracle.lightning_layer(3, 4, 3, [0.5, 0.9, 0.99],
                               mlp=oracle.moe(3, 2, 6, 0.7, (4, 1.0)))],
        streams=2, loop=(1, 3, 2))


CONFIGS = {"small": cfg_small, "ones": cfg_ones, "wide": cfg_wide,
           "tail": cfg_tail}


def make_engine(tmp_path, cfg, W, device, dtype="float32", blocks=48,
                block=4, slots=4, **kw):
    path = oracle.save_checkpoint(Path(tmp_path) / "ckpt", cfg, W)
    ecfg = EngineConfig(
        model=model_config_from_dir(path), block_size=block,
        num_gpu_blocks=blocks, max_num_seqs=slots,
        max_batched_tokens=kw.pop("max_batched_tokens", 4096),
        max_model_len=1024, use_hip_graphs=False,
        weights_path=path, dtype=dtype, **kw)
    return LLMEngine(ecfg, device=_dev(device))


def row_errors(got, ref):
    """Mean-free relative RMS difference per row, like a logit check."""
    got = torch.as_tensor(np.asarray(got.cpu() if torch.is_tensor(got)
                                     else got)).double()
    ref = torch.as_tensor(np.asarray(ref)).double()
    d = got - ref
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / ref.pow(2).mean().sqrt()


def close(got, ref, tol):
    err = row_errors(got, ref)
    assert float(err.max()) < tol, f"rel err {float(err.max()):.3e}"


def close_bf16(got, ref):
    """Rounding to bfloat16 can move a token across a router's choice;
    such rows are few."""
    err = row_errors(got, ref)
    assert float(err.median()) < 4e-2, f"median {float(err.median()):.3e}"
    assert float((err > 8e-2).double().mean()) < 0.1, err.sort()[0][-8:]


def toks(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def replay_all(engine, tokens, cuts):
    """Feed one request in portions `cuts`; logits of every position."""
    sid = engine.open_stream()
    out, at = [], 0
    for n in cuts:
        part = tokens[at:at + n]
        out.append(engine.replay_step([(sid, part)],
                                      {sid: list(range(len(part)))}))
        at += n
    assert at == len(tokens)
    engine.close_stream(sid)
    return torch.cat(out)


# ---------------------------------------------------------------------------
# mechanisms alone
# ---------------------------------------------------------------------------
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dims", [(1, 40), (2, 31), (3, 256), (4, 1024),
                                  (5, 1100), (8, 2052), (9, 64), (4, 8196)])
def test_stream_step(device, dims):
    """Three steps from the state after the embedding (one row in every
    stream): read only, write + read with a matrix that is far from
    symmetric, read through ones at the end."""
    B, D = dims
    g = torch.Generator().manual_seed(B * D)
    T, eps = 5, 1e-5
    x = torch.randn(T, D, generator=g)
    ys = [torch.randn(T, D, generator=g) for _ in range(2)]
    mix = [torch.randn(B, B, generator=g) for _ in range(2)]
    outw = [torch.randn(B, generator=g) for _ in range(2)]
    inw = [torch.randn(B, generator=g) for _ in range(2)] + [torch.ones(B)]
    w = torch.randn(D, generator=g)
    dev = _dev(device)
    X = np.stack([f64(x)] * B)
    s = x.to(dev).unsqueeze(1).expand(-1, B, -1)
    for n in range(3):
        if n:
            X = oracle.stream_update(X, f64(mix[n - 1]), f64(outw[n - 1]),
                                     f64(ys[n - 1]))
        want = oracle.rms_unit(oracle.stream_input(X, f64(inw[n])), eps) \
            * f64(w)
        s, h = ops.stream_step(
            s, ys[n - 1].to(dev) if n else None,
            mix[n - 1].to(dev) if n else None,
            outw[n - 1].to(dev) if n else None, inw[n].to(dev), w.to(dev),
            eps, torch.float32)
        np.testing.assert_allclose(f64(h), want, atol=2e-4, rtol=2e-4)
        np.testing.assert_allclose(f64(s).transpose(1, 0, 2), X, atol=1e-4,
                                   rtol=1e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_stream_step_bfloat16(device):
    g = torch.Generator().manual_seed(3)
    x = torch.randn(6, 4, 96, generator=g)
    y = torch.randn(6, 96, generator=g).bfloat16()
    mix, c, a = (torch.randn(*n, generator=g) for n in ((4, 4), (4,), (4,)))
    w = torch.rand(96, generator=g) + 0.5
    X = oracle.stream_update(f64(x).transpose(1, 0, 2), f64(mix), f64(c),
                             f64(y))
    want = oracle.rms_unit(oracle.stream_input(X, f64(a)), 1e-5) * f64(w)
    dev = _dev(device)
    s, h = ops.stream_step(x.to(dev), y.to(dev), mix.to(dev), c.to(dev),
                           a.to(dev), w.to(dev), 1e-5, torch.bfloat16)
    assert h.dtype == torch.bfloat16 and s.dtype == torch.float32
    np.testing.assert_allclose(f64(s).transpose(1, 0, 2), X, atol=1e-4)
    np.testing.assert_allclose(f64(h), want, atol=2e-2, rtol=1e-2)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dims", [(4, 2, 6, 4), (1, 1, 5, 2), (3, 3, 24, 24),
                                  (2, 1, 7, 6), (5, 5, 130, 66),
                                  (2, 2, 16, 6), (3, 1, 9, 0)])
def test_half_rotation_and_tied_values(device, dims):
    """Partial half-split rotation of queries and keys; the values in the
    cache are the keys before rotation."""
    H, G, N, rd = dims
    T, bs = 11, 4
    g = torch.Generator().manual_seed(N + rd)
    proj = torch.randn(T, (H + G) * N + 3, generator=g)
    pos = [0, 1, 2, 3, 4, 57, 58, 59, 1000, 1001, 12345]
    rot = {"dims": rd, "base": 400.0}
    x = f64(proj)
    q0 = x[:, :H * N].reshape(T, H, N)
    k0 = x[:, H * N:(H + G) * N].reshape(T, G, N)
    q_ref, k_ref = (oracle.rotate_halves(a, rot, pos) if rd else a
                    for a in (q0, k0))
    dev = _dev(device)
    kc = torch.zeros(6, G, bs, N, device=dev)
    vc = torch.zeros(6, G, bs, N, device=dev)
    slots = [5 * bs + 2, 5 * bs + 3, 1 * bs + 0] + list(range(8, 16))
    q = ops.qk_norm_rope_append(
        proj.to(dev), i32(pos, device), i32(slots, device), kc, vc, None,
        None, f32(oracle.rotary_frequencies(rot), device) if rd else None,
        1.0, 1e-5, H, G, N, N, half=True, tied=True)
    # fp32 angles: the error grows with the position
    tol = 2e-5 + 1.3e-7 * np.array(pos)[:, None, None] * 4
    assert (np.abs(f64(q).reshape(T, H, N) - q_ref) < tol).all()
    for t, s in enumerate(slots):
        assert (np.abs(f64(kc[s // bs, :, s % bs]) - k_ref[t])
                < tol[t]).all()
        np.testing.assert_allclose(f64(vc[s // bs, :, s % bs]), k0[t],
                                   atol=1e-6)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("half", [False, True])
@pytest.mark.parametrize("dims", [(4, 5, 4, 12), (1, 1, 2, 1), (3, 33, 20,
                                                               68),
                                  (7, 16, 64, 300)])
def test_latent_rope_append(device, half, dims):
    """Latent norm, rotation of the shared key and of every query head,
    append into scattered pages, either pair layout."""
    H, N, E, R = dims
    T, bs = 9, 4
    g = torch.Generator().manual_seed(N + R)
    x = torch.randn(T, H * (N + E) + R + E, generator=g)
    w = torch.rand(R, generator=g) + 0.5
    pos = [0, 1, 2, 60, 61, 62, 63, 64, 5000]
    rot = {"dims": E, "base": 90.0}
    turn = oracle.rotate_halves if half else oracle.rotate_neighbours
    d = f64(x)
    q_ref = d[:, :H * (N + E)].reshape(T, H, N + E).copy()
    q_ref[:, :, N:] = turn(q_ref[:, :, N:], rot, pos)
    c_ref = oracle.rms_unit(d[:, H * (N + E):-E], 1e-5) * f64(w)
    kr_ref = turn(d[:, None, -E:], rot, pos)[:, 0]
    dev = _dev(device)
    cache = torch.zeros(5, bs, R + E, device=dev)
    slots = [17, 18, 3] + list(range(8, 14))
    y = x.to(dev)
    ops.latent_rope_append(
        y, i32(pos, device), i32(slots, device), cache, w.to(dev),
        f32(oracle.rotary_frequencies(rot), device), 1e-5, H, N, E, R, half)
    tol = 3e-5 + 1.3e-7 * np.array(pos)[:, None] * 4
    got = f64(y)[:, :H * (N + E)].reshape(T, H, N + E)
    assert (np.abs(got - q_ref) < tol[:, :, None]).all()
    rows = f64(cache).reshape(-1, R + E)[slots]
    np.testing.assert_allclose(rows[:, :R], c_ref, atol=3e-5)
    assert (np.abs(rows[:, R:] - kr_ref) < tol).all()


class SinkCase:
    """One sequence's queries, rotated keys and tied values in scattered
    pages."""

    def __init__(self, device, dtype, H, G, N, bs, ctx, seed=0):
        g = torch.Generator().manual_seed(ctx + N + seed)
        self.device, self.bs, self.dtype = _dev(device), bs, dtype
        rnd = lambda *s: torch.randn(*s, generator=g).to(dtype)  # noqa: E731
        self.q, self.k, self.v = rnd(ctx, H, N), rnd(ctx, G, N), rnd(ctx, G,
                                                                    N)
        self.sink = torch.randn(H, generator=g) * 2.0
        nb = (ctx + bs - 1) // bs
        self.perm = torch.randperm(nb + 2, generator=g)[:nb].tolist()
        self.nb = nb

    def reference(self, scale):
        return oracle.sink_attention(f64(self.q), f64(self.k), f64(self.v),
                                     scale, f64(self.sink))

    def run(self, scale, rows=None):
        dev, ctx = self.device, len(self.k)
        G, N = self.k.shape[1:]
        kc, vc = (torch.zeros(self.nb + 2, G, self.bs, N, dtype=self.dtype,
                              device=dev) for _ in range(2))
        for j in range(ctx):
            b, o = self.perm[j // self.bs], j % self.bs
            kc[b, :, o], vc[b, :, o] = self.k[j].to(dev), self.v[j].to(dev)
        sel = list(range(ctx)) if rows is None else rows
        n = len(sel)
        q = self.q[sel].reshape(n, -1).to(dev)
        if rows is None:
            seq = dict(num_prefill_rows=n, prefill_seq_lens=[n],
                       seq_cu=i32([0, n], dev), seq_start=i32([0], dev))
            bt, rs = i32([self.perm], dev), i32([0] * n, dev)
        else:
            seq = dict(num_prefill_rows=0, prefill_seq_lens=None,
                       seq_cu=i32(list(range(n + 1)), dev),
                       seq_start=i32(sel, dev))
            bt, rs = i32([self.perm] * n, dev), i32(list(range(n)), dev)
        o = ops.softcap_attention(q, kc, vc, bt, rs, i32(sel, dev), scale,
                                  sinks=self.sink.to(dev), **seq)
        return f64(o.float()).reshape(n, -1, N)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dims", [(4, 2, 6, 4), (1, 1, 1, 2), (3, 3, 17, 8),
                                  (6, 1, 66, 4)])
def test_sinks_and_far_keys(device, dims):
    """Learned sinks that differ per head; then one key at every page
    border that stands out for the last query; then scores so low that
    the sinks take nearly all the weight."""
    H, G, N, bs = dims
    ctx = 53
    c = SinkCase(device, torch.float32, H, G, N, bs, ctx)
    ref = c.reference(0.3)
    np.testing.assert_allclose(c.run(0.3), ref, atol=5e-5, rtol=5e-5)
    rows = [0, 1, bs - 1, bs, 30, 52]
    np.testing.assert_allclose(c.run(0.3, rows), ref[rows], atol=5e-5)
    for j in (0, 1, bs - 1, bs, 2 * bs - 1, 2 * bs, 51):
        c = SinkCase(device, torch.float32, H, G, N, bs, ctx, seed=j)
        c.q[52, :] = c.q[52, 0] / c.q[52, 0].norm() * 5.0
        c.k[j, :] = c.q[52, 0] * 2.0
        ref = c.reference(1.0)
        # the boosted key decides the last row
        assert np.abs(ref[52] - f64(c.v[j]).repeat(H // G, 0)).max() < 1e-3
        np.testing.assert_allclose(c.run(1.0), ref, atol=1e-4)
        np.testing.assert_allclose(c.run(1.0, [52]), ref[52:], atol=1e-4)
    c.q *= 0.0
    c.sink = torch.linspace(6.0, 9.0, H)
    ref = c.reference(1.0)
    assert np.abs(ref[0]).max() < 0.05
    np.testing.assert_allclose(c.run(1.0), ref, atol=1e-5)


@pytest.mark.gpu
@pytest.mark.parametrize("dims", [(4, 2, 64, 16), (9, 3, 88, 16),
                                  (8, 1, 128, 8), (6, 6, 24, 16)])
def test_sink_attention_tile_kernel_bf16(dims):
    H, G, N, bs = dims
    c = SinkCase("cuda", torch.bfloat16, H, G, N, bs, 210)
    ref = c.reference(N ** -0.5)
    assert np.abs(c.run(N ** -0.5) - ref).max() < 0.06
    rows = [0, 3, 63, 64, 65, 128, 200, 209]
    assert np.abs(c.run(N ** -0.5, rows) - ref[rows]).max() < 0.06


class DecayCase:
    """Unequal sequences in slots of a state buffer full of garbage, in
    several steps."""

    def __init__(self, device, dtype, H, G, N, P, lens, decay=None, seed=0):
        g = torch.Generator().manual_seed(N + P + seed)
        self.device, self.dtype = _dev(device), dtype
        self.H, self.G, self.N, self.P = H, G, N, P
        self.decay = torch.linspace(0.35, 1.0, H) if decay is None \
            else torch.tensor(decay)
        self.seqs = [tuple(torch.randn(*s, generator=g).to(dtype)
                           for s in ((L, G, N), (L, G, N), (L, H, P)))
                     for L in lens]
        self.state = torch.randn(len(lens) + 2, H * N * P,
                                 generator=g).to(self.device)
        self.slots = torch.randperm(len(lens) + 2,
                                    generator=g)[:len(lens)].tolist()

    def reference(self, s, rounded=False):
        """rounded: silu results as the activation type holds them."""
        def act(x):
            y = oracle.silu(f64(x))
            return f64(torch.from_numpy(y).to(self.dtype)) if rounded else y
        q, k, v = (act(x) for x in self.seqs[s])
        rep = self.H // self.G
        return oracle.decayed_memory(np.repeat(q, rep, 1),
                                     np.repeat(k, rep, 1), v,
                                     f64(self.decay))

    def step(self, plan):
        """plan: [(sequence, first row, rows)].  The projections arrive
        as strided views of one fused matrix."""
        H, G, N, P = self.H, self.G, self.N, self.P
        rows = [n for _s, _a, n in plan]
        cu = np.concatenate([[0], np.cumsum(rows)]).tolist()
        fused = torch.cat([torch.cat(
            [x[a:a + n].reshape(n, -1) for x in self.seqs[s]], 1)
            for s, a, n in plan])
        fused = torch.nn.functional.pad(fused, (0, 8)).to(self.device)
        T = cu[-1]
        q0, k0, v0 = 0, G * N, 2 * G * N
        return ops.fixed_decay_scan(
            fused[:, q0:k0].view(T, G, N), fused[:, k0:v0].view(T, G, N),
            fused[:, v0:v0 + H * P].view(T, H, P),
            self.decay.to(self.device), self.state, i32(cu, self.device),
            i32([a for _s, a, _n in plan], self.device),
            i32([self.slots[s] for s, _a, _n in plan], self.device), rows)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dims", [(2, 1, 5, 7), (3, 3, 16, 64), (1, 1, 1, 1),
                                  (2, 2, 40, 70), (2, 1, 150, 132)])
def test_fixed_decay_steps(device, dims):
    """A fresh sequence over a stale slot, a continued one, a one-row one
    and one left out of a step; 32-bit."""
    c = DecayCase(device, torch.float32, *dims, [41, 9, 1, 6])
    refs = [c.reference(s) for s in range(4)]
    for plan in ([(0, 0, 19), (1, 0, 2), (2, 0, 1)],
                 [(1, 2, 1), (3, 0, 5), (0, 19, 1)],
                 [(0, 20, 21), (3, 5, 1), (1, 3, 6)]):
        out = f64(c.step(plan))
        want = np.concatenate([refs[s][0][a:a + n] for s, a, n in plan])
        np.testing.assert_allclose(out, want, atol=3e-5 * np.abs(want).max(),
                                   rtol=3e-5)
    for s in range(4):
        end = refs[s][1]
        np.testing.assert_allclose(
            f64(c.state[c.slots[s]]).reshape(end.shape), end,
            atol=3e-5 * max(1.0, np.abs(end).max()), rtol=3e-5)


@pytest.mark.parametrize("device", DEVICES)
def test_decay_reaches_exactly_one_step(device):
    """The memory before row t decays once on the way to t and the row's
    own key not at all; the first row of a reused slot sees no memory."""
    big = 20.0                                # silu(20) = 20 to 4e-8
    q = torch.full((1, 1, 1), big)
    c = DecayCase(device, torch.float32, 1, 1, 1, 1, [3], decay=[0.25])
    c.seqs[0] = (torch.full((3, 1, 1), big),
                 torch.tensor([big, -400.0, -400.0]).view(3, 1, 1),
                 torch.full((3, 1, 1), big))
    del q
    got = torch.cat([c.step([(0, t, 1)]) for t in range(3)]).view(-1)
    want = big ** 3 * 0.25 ** np.arange(3)
    np.testing.assert_allclose(f64(got), want, rtol=1e-5)


@pytest.mark.gpu
@pytest.mark.parametrize("dims", [
    (2, 2, 32, 64), (3, 1, 64, 48), (2, 1, 128, 128), (2, 2, 24, 200),
    (4, 4, 40, 72), (1, 1, 1, 1), (2, 2, 13, 9), (2, 1, 96, 130)])
def test_fixed_decay_chunks_bf16(dims):
    """MFMA chunks: unequal sequences, chunk edges, partial chunks, rows
    that continue a state, a mix with the step kernel; strong and absent
    decay.  Against rounded activations the recurrence itself is exact to
    far below bfloat16."""
    H = dims[0]
    c = DecayCase("cuda", torch.bfloat16, *dims, [200, 64, 65, 17, 3],
                  decay=[0.02, 1.0, 0.9, 0.5][:H])
    refs = [c.reference(s, rounded=True) for s in range(5)]
    for plan in ([(0, 0, 129), (1, 0, 64), (2, 0, 1), (3, 0, 16)],
                 [(2, 1, 64), (4, 0, 2), (0, 129, 1)],
                 [(0, 130, 70), (3, 16, 1), (4, 2, 1)]):
        out = f64(c.step(plan))
        want = np.concatenate([refs[s][0][a:a + n] for s, a, n in plan])
        # each head against its own scale: strongly decayed heads are small
        err = np.abs(out - want).max((0, 2))
        assert (err < 2e-3 * np.abs(want).max((0, 2)) + 1e-6).all(), err
        rms = np.sqrt(((out - want) ** 2).mean() / (want ** 2).mean())
        assert rms < 3e-4, rms
    for s in range(5):
        end = refs[s][1]
        got = f64(c.state[c.slots[s]]).reshape(end.shape)
        assert np.abs(got - end).max() < 1e-3 * max(1.0, np.abs(end).max())


@pytest.mark.gpu
@pytest.mark.parametrize("dims", [(2, 2, 64, 64), (3, 1, 128, 136)])
def test_fixed_decay_segments_bf16(dims):
    """Few long sequences are cut into segments that run side by side:
    same read-outs and state as one after the other, from a fresh and
    from a continued memory."""
    c = DecayCase("cuda", torch.bfloat16, *dims, [1500, 700],
                  decay=[0.999, 1.0, 0.97][:dims[0]])
    refs = [c.reference(s, rounded=True) for s in range(2)]
    for plan in ([(0, 0, 700), (1, 0, 650)], [(0, 700, 800), (1, 650, 50)]):
        _s, segs, first = ops._decay_plan(
            tuple(n for _q, _a, n in plan),
            dims[0] * -(-dims[3] // 128), True, c.state.device)
        assert first is not None and segs.shape[1] > 2
        out = f64(c.step(plan))
        want = np.concatenate([refs[s][0][a:a + n] for s, a, n in plan])
        rms = np.sqrt(((out - want) ** 2).mean((0, 2))
                      / (want ** 2).mean((0, 2)))
        assert rms.max() < 3e-4, rms
    for s in range(2):
        end = refs[s][1]
        got = f64(c.state[c.slots[s]]).reshape(end.shape)
        assert np.abs(got - end).max() < 1e-3 * np.abs(end).max()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dims", [(3, 24, 1), (5, 7, 1), (18, 64, 1),
                                  (12, 200, 2), (10, 300, 1), (16, 512, 1),
                                  (3, 401, 1), (20, 512, 1)])
def test_read_out_norm_over_many_channels(device, dims):
    """One RMS norm over all heads together, or over half of them, times
    the weight and the gate, with and without a normaliser per head."""
    H, P, parts = dims
    C = H * P
    g = torch.Generator().manual_seed(C)
    o = torch.randn(5, H, P, generator=g) * 3.0
    gate = torch.randn(5, C + 8, generator=g)[:, :C]
    w = torch.randn(C, generator=g)
    den = torch.randn(5, H, generator=g)
    dev = _dev(device)
    for d, first, kind in ((None, False, ops.GATE_SIGMOID),
                           (den, True, ops.GATE_SILU)):
        a = f64(gate)
        a = oracle.silu(a) if kind == ops.GATE_SILU else oracle.sigmoid(a)
        y = f64(o)
        if d is not None:
            y = y / (np.abs(f64(d)) + 1e-6)[:, :, None]
        y = y.reshape(5, C) * (a if first else 1.0)
        y = oracle.rms_unit(y.reshape(5, parts, -1), 1e-5).reshape(5, C) \
            * f64(w) * (1.0 if first else a)
        got = ops.head_norm_gate(
            o.to(dev), gate.to(dev), w.to(dev), 1e-5, C // parts, kind,
            first, None if d is None else d.to(dev), None, torch.float32)
        np.testing.assert_allclose(f64(got), y, atol=3e-5, rtol=1e-4)


def test_decay_plan_covers_every_row_once():
    for rows in ((700,), (16, 15, 0, 64), (1, 1, 1), (5000, 3, 20),
                 (256, 256, 255)):
        for blocks in (1, 8, 300):
            short, segs, first = ops._decay_plan(rows, blocks, True, "cpu")
            seen = [0] * sum(rows)
            cu = np.concatenate([[0], np.cumsum(rows)])
            for s in ([] if short is None else short.tolist()):
                assert 0 < rows[s] < ops.FIXED_DECAY_CHUNKS_FROM
                for r in range(cu[s], cu[s + 1]):
                    seen[r] += 1
            tab = [] if segs is None else segs.t().tolist()
            for n, (a, b, s, f, l) in enumerate(tab):
                assert cu[s] <= a < b <= cu[s + 1]
                assert f == (a == cu[s]) and l == (b == cu[s + 1])
                for r in range(a, b):
                    seen[r] += 1
            assert seen == [1] * len(seen)
            if first is not None:
                f = first.tolist()
                assert f[0] == 0 and f[-1] == len(tab)
                for a, b in zip(f, f[1:]):
                    assert len({t[2] for t in tab[a:b]}) == 1


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("shape", [(8, 3), (1, 1), (5, 5), (64, 8), (13, 2)])
def test_softmax_router(device, shape):
    """Weights are entries of the softmax over ALL experts: they do not
    sum to one unless every expert is chosen.  Logits are a strided view
    (the shared expert's gate sits behind them)."""
    E, K = shape
    g = torch.Generator().manual_seed(E * K)
    logits = torch.randn(50, E + 1, generator=g) * 2.0
    w, idx, dst = ops.moe_topk_route(logits.to(_dev(device))[:, :E], K, 64,
                                     over_all=True)
    idx, w = idx.cpu().tolist(), w.cpu()
    for t in range(50):
        want = dict(oracle.route(f64(logits[t, :E]), K))
        assert sorted(idx[t]) == sorted(want)
        for e, x in zip(idx[t], w[t].tolist()):
            assert abs(x - want[e]) < 1e-6
    assert K == E or float(w.sum(1).max()) < 1.0
    if dst is not None:
        d = dst.cpu().tolist()
        assert len(set(d)) == len(d)
        flat = [e for row in idx for e in row]
        assert all(e * 64 <= r < e * 64 + 50 for e, r in zip(flat, d))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("shared", [False, True])
@pytest.mark.parametrize("dims", [(7, 3, 6, 20), (1, 1, 1, 9),
                                  (300, 2, 5, 64)])
def test_expert_dispatch_both_routes(device, shared, dims):
    """Padded and sorted dispatch against the sum written out, with and
    without the gated shared rows."""
    T, K, E, D = dims
    g = torch.Generator().manual_seed(T + D)
    x = torch.randn(T, D, generator=g)
    up = torch.randn(E, D, D, generator=g) * D ** -0.5
    down = torch.randn(E, D, D, generator=g) * D ** -0.5
    logits = torch.randn(T, E + 1, generator=g)
    sh = torch.randn(T, D, generator=g) if shared else None
    dev = _dev(device)
    C = (T + 63) // 64 * 64
    w, idx, dst = ops.moe_topk_route(logits.to(dev)[:, :E], K, C,
                                     over_all=True)
    if dst is None:
        dst = moe_common.padded_rows(idx, E, C)
    want = np.zeros((T, D))
    for t in range(T):
        for e, a in oracle.route(f64(logits[t, :E]), K):
            want[t] += a * (np.maximum(f64(x[t]) @ f64(up[e]), 0.0)
                            @ f64(down[e]))
    if shared:
        want += oracle.sigmoid(f64(logits[:, E:])) * f64(sh)
    for rows in (dst, None):
        out = moe_common.experts_combined(
            x.to(dev), w, idx, rows, C, up.to(dev), down.to(dev),
            torch.relu, None if sh is None else sh.to(dev),
            logits.to(dev)[:, E] if shared else None)
        np.testing.assert_allclose(f64(out), want, atol=2e-5, rtol=2e-5)


@pytest.mark.parametrize("device", DEVICES)
def test_expert_limits_are_their_own(tmp_path, device):
    """Routed and shared experts clamp at different limits, the gate from
    above only: inputs far outside either limit."""
    f = oracle.moe(3, 2, 7, 0.4, (5, 1.7))
    cfg = oracle.make_config(12, 19, [
        oracle.attention_layer(1, 1, 4, 2, 10.0, 0.5, mlp=f)])
    W = oracle.random_weights(cfg, 5)
    for n in W:
        if n.endswith((".gate", ".up")):
            W[n] = W[n] * 8.0
    eng = make_engine(tmp_path, cfg, W, device)
    h = np.random.default_rng(1).normal(size=(9, 12))
    want = oracle.moe_ff(h, W, "l0.mlp.", f)
    mlp = eng.model.layers[0].mlp
    assert (mlp.spec.limit, mlp.spec.shared_limit) == (0.4, 1.7)
    got = mlp(f32(h, device), None)
    np.testing.assert_allclose(f64(got), want, atol=1e-4, rtol=1e-4)


# ---------------------------------------------------------------------------
# the engine against the oracle
# ---------------------------------------------------------------------------
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_prompt_layers_and_logits(tmp_path, device, name):
    cfg = CONFIGS[name]()
    W = oracle.random_weights(cfg, 11)
    eng = make_engine(tmp_path, cfg, W, device)
    t = toks(41, cfg["vocab"], 12)
    ref, taps_ref = oracle.forward(W, cfg, t)
    taps = []
    eng.model.tap = lambda i, x: taps.append(f64(x))
    got = replay_all(eng, t, [41])
    eng.model.tap = None
    assert len(taps) == len(oracle.layer_runs(cfg))
    for i, (a, b) in enumerate(zip(taps, taps_ref)):
        assert np.abs(a - b).max() < 2e-4 * max(1.0, np.abs(b).max()), i
    close(got, ref, 2e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_portions_and_token_by_token(tmp_path, device, name):
    """The same request whole, token by token, and in ragged portions
    down to two tokens; slots and pages are reused from run to run."""
    cfg = CONFIGS[name]()
    W = oracle.random_weights(cfg, 13)
    eng = make_engine(tmp_path, cfg, W, device, blocks=16)
    t = toks(37, cfg["vocab"], 14)
    ref, _ = oracle.forward(W, cfg, t)
    for cuts in ([37], [1] * 37, [2, 2, 5, 1, 1, 9, 2, 3, 12],
                 [30] + [1] * 7, [3, 1, 33], [2] * 18 + [1]):
        close(replay_all(eng, t, cuts), ref, 2e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_mixed_batches_against_each_alone(tmp_path, device):
    """Four unequal requests interleaved (portions beside single
    tokens, a request left out of steps, a fifth admitted into a freed
    slot and freed pages) give what each gives alone."""
    cfg = cfg_small()
    W = oracle.random_weights(cfg, 15)
    eng = make_engine(tmp_path, cfg, W, device, blocks=36, slots=4)
    reqs = {n: toks(L, cfg["vocab"], 20 + i) for i, (n, L) in enumerate(
        [("a", 50), ("b", 23), ("c", 9), ("d", 31), ("e", 17)])}
    ref = {n: oracle.forward(W, cfg, t)[0] for n, t in reqs.items()}
    plan = [
        {"a": 3, "b": 3},
        {"a": 20, "c": 2},
        {"a": 1, "b": 17, "c": 1, "d": 2},
        {"a": 2, "c": 6, "d": 16},
        {"b": 1, "d": 1},
        {"a": 1, "b": 1, "d": 1},
        {"a": 13, "b": 1, "d": 11, "e": 5},     # e takes c's slot
        {"a": 10, "e": 1},
        {"e": 11},
    ]
    ids, at, got = {}, {n: 0 for n in reqs}, {n: [] for n in reqs}
    for step in plan:
        feeds, want = [], {}
        for n, k in step.items():
            if n not in ids:
                ids[n] = eng.open_stream()
            part = reqs[n][at[n]:at[n] + k]
            feeds.append((ids[n], part))
            want[ids[n]] = list(range(k))
            at[n] += k
        out = eng.replay_step(feeds, want)
        r = 0
        for n, k in step.items():
            got[n].append(out[r:r + k])
            r += k
        for n in list(step):
            if at[n] == len(reqs[n]):
                eng.close_stream(ids[n])
    for n in reqs:
        assert at[n] == len(reqs[n])
        close(torch.cat(got[n]), ref[n], 2e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_first_tokens_in_used_slots(tmp_path, device):
    """Requests of one, two and three tokens in slots and pages that
    longer requests have just left: nothing of the old memories, keys and
    latents shows."""
    cfg = cfg_small()
    W = oracle.random_weights(cfg, 61)
    eng = make_engine(tmp_path, cfg, W, device, blocks=24, slots=3)
    for n in (19, 23, 11):                     # dirty every slot and page
        replay_all(eng, toks(n, cfg["vocab"], 60 + n), [n])
    reqs = [toks(n, cfg["vocab"], 70 + n) for n in (1, 2, 3)]
    refs = [oracle.forward(W, cfg, t)[0] for t in reqs]
    ids = [eng.open_stream() for _ in reqs]
    out = eng.replay_step(
        [(i, t[:2]) for i, t in zip(ids, reqs)],
        {i: list(range(min(2, len(t)))) for i, t in zip(ids, reqs)})
    close(out, np.concatenate([r[:2] for r in refs]), 2e-4)
    out = eng.replay_step([(ids[2], reqs[2][2:])], {ids[2]: [0]})
    close(out, refs[2][2:], 2e-4)
    for i in ids:
        eng.close_stream(i)


@pytest.mark.parametrize("device", DEVICES)
def test_every_pass_of_the_loop_has_its_own_cache(tmp_path, device):
    """Buffers per layer run, all distinct; the oracle moves when the
    loop runs once more or once less."""
    cfg = cfg_small()
    W = oracle.random_weights(cfg, 33)
    eng = make_engine(tmp_path, cfg, W, device)
    runs = oracle.layer_runs(cfg)
    assert runs == [0, 1, 2, 1, 2, 1, 2, 3]
    assert len(eng.kv_caches) == len(runs)
    ptrs = [t.data_ptr() for t, _k in eng.kv_caches._all()]
    assert len(set(ptrs)) == len(ptrs)
    # latent, then (K and V, memory) x 3, then K and V
    assert len(ptrs) == 1 + 3 * 3 + 2
    t = toks(30, cfg["vocab"], 34)
    ref, _ = oracle.forward(W, cfg, t)
    for times in (2, 4):
        other = json.loads(json.dumps(cfg))
        other["loop"]["times"] = times
        assert np.abs(oracle.forward(W, other, t)[0] - ref).max() > 1e-2
    close(replay_all(eng, t, [13, 1, 2, 14]), ref, 2e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_long_decode(tmp_path, device):
    cfg = cfg_small()
    W = oracle.random_weights(cfg, 16)
    eng = make_engine(tmp_path, cfg, W, device, blocks=80)
    t = toks(230, cfg["vocab"], 17)
    ref, _ = oracle.forward(W, cfg, t)
    close(replay_all(eng, t, [6] + [1] * 224), ref, 3e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind", ["attention", "latent", "lightning"])
def test_far_token_reaches_the_logits(tmp_path, device, kind):
    """Weights that make one far token decisive for the last query, in a
    prompt and decoded: the engine follows the oracle, and the oracle
    moves when the far token is another."""
    if kind == "attention":
        layer = oracle.attention_layer(2, 1, 8, 2, 1e6, 6.0)
    elif kind == "latent":
        layer = oracle.latent_layer(2, 8, 2, 8, 8, 1e6, 6.0)
    else:
        layer = oracle.lightning_layer(2, 8, 8, [1.0, 0.999])
    cfg = oracle.make_config(32, 41, [layer], streams=2)
    W = oracle.random_weights(cfg, 71)
    W["embed"][7], W["embed"][9] = 0.0, 0.0
    W["embed"][7, 0] = W["embed"][9, 1] = 6.0
    # token 7 leaves a key on entry 5 of the head that nothing else has,
    # token 9's query asks for it
    key = "l0.mix." + ("dkv" if kind == "latent" else "k")
    W[key][5] = 0.0
    W[key][5, 0] = 4.0
    W["l0.mix.q"][5] *= 0.125
    W["l0.mix.q"][5, 1] = 6.0
    if kind == "latent":
        W["l0.mix.uk"][:] = 0.0
        W["l0.mix.uk"][5, 5] = 2.0
    if kind != "lightning":
        W["l0.mix.sink"][:] = 0.5
    t = [x if x not in (7, 9) else 8 for x in toks(120, 41, 72)]
    t[17], t[60], t[119] = 7, 9, 9
    ref, _ = oracle.forward(W, cfg, t)
    u = list(t)
    u[17] = 8
    moved = np.abs(oracle.forward(W, cfg, u)[0] - ref)
    assert moved[119].max() > 2e-2 and moved[:17].max() < 1e-12
    eng = make_engine(tmp_path, cfg, W, device)
    close(replay_all(eng, t, [120]), ref, 2e-4)
    close(replay_all(eng, t, [17, 1, 70, 2, 7] + [1] * 23), ref, 2e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_bfloat16_mode(tmp_path, device):
    cfg = cfg_small()
    W = oracle.random_weights(cfg, 18)
    eng = make_engine(tmp_path, cfg, W, device, dtype="bfloat16")
    t = toks(33, cfg["vocab"], 19)
    ref, _ = oracle.forward(W, cfg, t)
    close_bf16(replay_all(eng, t, [33]), ref)
    close_bf16(replay_all(eng, t, [5, 2, 1, 1, 20, 4]), ref)


@pytest.mark.gpu
def test_bfloat16_tile_sizes_through_the_engine(tmp_path):
    """Head, latent and memory sizes that take the MFMA paths, a prompt
    of several tiles and chunks, both expert routes, portions and decoded
    rows, in bfloat16."""
    cfg = oracle.make_config(128, 97, [
        oracle.attention_layer(6, 2, 48, 24, 10000.0, 0.15,
                               mlp=oracle.moe(6, 2, 56, 1.4, (72, 2.2))),
        oracle.lightning_layer(3, 40, 56, [0.7, 0.96, 0.999],
                               mlp=oracle.dense(200)),
        oracle.latent_layer(6, 40, 24, 32, 88, 10000.0, 0.125,
                            mlp=oracle.dense(160))],
        streams=4, loop=(1, 2, 2))
    W = oracle.random_weights(cfg, 51)
    eng = make_engine(tmp_path, cfg, W, "cuda", dtype="bfloat16", blocks=60,
                      block=16)
    t = toks(300, cfg["vocab"], 52)
    ref, _ = oracle.forward(W, cfg, t)
    close_bf16(replay_all(eng, t, [300]), ref)
    close_bf16(replay_all(eng, t, [70, 2, 200, 1, 1, 26]), ref)


def _greedy(cfg, W, prompt, n):
    t = list(prompt)
    for _ in range(n):
        t.append(int(np.argmax(oracle.forward(W, cfg, t)[0][-1])))
    return t[len(prompt):]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("mode", ["plain", "chunked_mixed"])
def test_greedy_generation_through_scheduler(tmp_path, device, mode):
    cfg = cfg_small()
    W = oracle.random_weights(cfg, 21)
    kw = {}
    if mode == "chunked_mixed":
        kw = dict(enable_chunked_prefill=True, enable_mixed_batches=True,
                  max_batched_tokens=7)
    eng = make_engine(tmp_path, cfg, W, device, **kw)
    prompts = [toks(n, cfg["vocab"], 30 + n) for n in (5, 19, 11)]
    sp = SamplingParams(max_new_tokens=6, temperature=0.0)
    rids = [eng.add_request(p, sp) for p in prompts]
    for _ in range(200):
        if eng.is_finished():
            break
        eng.step()
    for rid, p in zip(rids, prompts):
        assert eng.get_output(rid).token_ids == _greedy(cfg, W, p, 6)


@pytest.mark.parametrize("device", DEVICES)
def test_preemption_restarts_every_state(tmp_path, device):
    """A pool too small for both requests: the newer one is preempted
    and resumes by re-running its folded prompt."""
    cfg = cfg_small()
    W = oracle.random_weights(cfg, 26)
    prompts = [toks(7, cfg["vocab"], 41), toks(6, cfg["vocab"], 42)]
    refs = [_greedy(cfg, W, p, 10) for p in prompts]
    eng = make_engine(tmp_path, cfg, W, device, blocks=8, block=4)
    sp = SamplingParams(max_new_tokens=10, temperature=0.0)
    ids = [eng.add_request(p, sp) for p in prompts]
    for _ in range(300):
        if eng.is_finished():
            break
        eng.step()
    assert eng.scheduler.num_preemptions > 0
    for i, r in zip(ids, refs):
        assert eng.get_output(i).token_ids == r


@pytest.mark.parametrize("device", DEVICES)
def test_forked_group_copies_pages_and_memories(tmp_path, device):
    """n=2 from one prefill: the branch shares the prompt's full pages
    and gets a copy of the partial one and of every pass's memory."""
    cfg = cfg_small()
    W = oracle.random_weights(cfg, 27)
    prompt = toks(10, cfg["vocab"], 43)     # 2 full pages + a partial one
    ref = _greedy(cfg, W, prompt, 5)
    eng = make_engine(tmp_path, cfg, W, device, blocks=32)
    ids = eng.add_request_group(
        prompt, SamplingParams(max_new_tokens=5, temperature=0.0), n=2)
    while not eng.is_finished():
        eng.step()
    assert eng.num_forks == 1
    for i in ids:
        assert eng.get_output(i).token_ids == ref


def test_registry_config_and_loader_errors(tmp_path):
    cfg = cfg_small()
    W = oracle.random_weights(cfg, 22)
    path = oracle.save_checkpoint(tmp_path / "m", cfg, W)
    mc = model_config_from_dir(path)
    assert isinstance(mc, DefosunConfig) and is_recurrent(mc) and mc.is_moe
    assert [l.type for l in mc.layers] == ["latent_attention", "attention",
                                           "lightning", "attention"]
    assert mc.layer_runs == [0, 1, 2, 1, 2, 1, 2, 3] and mc.streams == 3
    a, d, f = mc.layers[1].mixer, mc.layers[2].mixer, mc.layers[0].mlp
    assert a.tied_values and a.rot_half and not a.qk_norm and a.out_bias
    assert d.decay == (0.3, 0.8, 0.97, 1.0, 0.55)
    assert (f.limit, f.shared_limit, f.shared_ff, f.top) == (1.1, 0.6, 9, 3)
    assert mc.layers[2].mlp.shared_ff == 0 and mc.layers[3].mlp is None
    # keys and values of every pass, latent rows
    assert mc.kv_bytes_per_token(2) == 2 * (
        (12 + 4) + 3 * 2 * (10 + 10) + 3 * (8 + 8))
    assert not is_recurrent(DefosunConfig.from_dict(oracle.make_config(
        8, 9, [oracle.attention_layer(1, 1, 4, 2, 10.0, 0.5)])))
    # sizes come from the tensors when the json has none
    bare = json.loads(json.dumps(cfg))
    del bare["layers"][0]["mixer"]["kv_rank"]
    del bare["layers"][0]["mlp"]["router"]["experts"]
    del bare["layers"][0]["mlp"]["expert"]["ff"]
    del bare["layers"][0]["mlp"]["shared"]["ff"]
    del bare["layers"][1]["mlp"]["ff"]
    p2 = oracle.save_checkpoint(tmp_path / "m2", bare, W)
    assert model_config_from_dir(p2).layers == mc.layers
    bad = dict(W)
    bad["l0.mix.dkv"] = bad["l0.mix.dkv"][:-1]
    with pytest.raises(ValueError, match="l0.mix.q"):
        make_engine(tmp_path / "e", cfg, bad, "cpu")
    with pytest.raises(ValueError, match="unknown mixer"):
        DefosunConfig.from_dict(oracle.make_config(
            8, 9, [{"type": "lstm", "mixer": {}, "mlp": None}]))
    with pytest.raises(ValueError, match="unknown mlp"):
        DefosunConfig.from_dict(oracle.make_config(8, 9, [
            oracle.attention_layer(1, 1, 4, 2, 10.0, 0.5,
                                   mlp={"kind": "conv"})]))
    with pytest.raises(ValueError, match="decays"):
        DefosunConfig.from_dict(oracle.make_config(8, 9, [
            oracle.lightning_layer(2, 4, 4, [0.5])]))
    with pytest.raises(ValueError, match="loop"):
        DefosunConfig.from_dict(oracle.make_config(8, 9, [
            oracle.attention_layer(1, 1, 4, 2, 10.0, 0.5)], loop=(0, 2, 2)))
    with pytest.raises(ValueError, match="keys' width"):
        c = oracle.make_config(8, 9, [
            oracle.attention_layer(1, 1, 4, 2, 10.0, 0.5)])
        c["layers"][0]["mixer"]["vdim"] = 6
        DefosunConfig.from_dict(c)


def test_preset_runs_and_forks_copy_state():
    eng = LLMEngine(EngineConfig.tiny_defosun(), device="cpu")
    rid = eng.add_request(list(range(1, 20)),
                          SamplingParams(max_new_tokens=4, temperature=0.0))
    while not eng.is_finished():
        eng.step()
    assert len(eng.get_output(rid).token_ids) == 4
    mem = eng.kv_caches[1]
    mem[2].fill_(3.0)
    eng.kv_caches.copy_slot(2, 0)
    assert torch.equal(mem[0], mem[2])


def test_local_provider_serves_a_checkpoint_directory(tmp_path):
    """The gateway's local provider with LOCAL_MODEL=hf picks the
    architecture from the directory's config.json and generates through
    the async engine with sampling."""
    import asyncio

    from inference_gateway_amd.config import LocalConfig
    from inference_gateway_amd.providers.local import LocalProvider

    cfg = oracle.make_config(48, 300, [
        oracle.attention_layer(2, 1, 8, 4, 100.0, 0.35,
                               mlp=oracle.dense(32)),
        oracle.lightning_layer(2, 8, 10, [0.9, 0.5],
                               mlp=oracle.moe(4, 2, 16, 1.0, (8, 1.5)))],
        loop=(0, 2, 2))
    W = oracle.random_weights(cfg, 35)
    path = oracle.save_checkpoint(tmp_path / "m", cfg, W)
    lc = LocalConfig(enabled=True, model="hf", max_num_seqs=4,
                     max_model_len=128)
    lc.num_gpu_blocks = 64
    lc.weights_path = path
    provider = LocalProvider(lc, device="cpu")
    try:
        assert isinstance(provider.engine.engine.cfg.model, DefosunConfig)

        async def go(temp):
            return await provider.chat_completions({
                "model": "local/hf",
                "messages": [{"role": "user", "content": "hi"}],
                "max_tokens": 3, "temperature": temp, "top_p": 0.9})

        assert asyncio.run(go(0))["usage"]["completion_tokens"] == 3
        assert asyncio.run(go(0.8))["usage"]["completion_tokens"] == 3
    finally:
        provider.engine.shutdown()


def test_trace_command(tmp_path):
    """bin/trace_run end to end on a small checkpoint: portions, a
    decoded token, a step with nothing wanted, a second request that
    reuses the first one's slot."""
    cfg = cfg_tail()
    W = oracle.random_weights(cfg, 23)
    path = oracle.save_checkpoint(tmp_path / "m", cfg, W)
    a, b = toks(9, cfg["vocab"], 24), toks(4, cfg["vocab"], 25)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:5],
                                 "want": [0, 4]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": a[5:8], "want": []}],
         "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": a[8:], "want": [0]},
                                {"id": "b", "tokens": b, "want": [3]}],
         "end": ["a", "b"]},
    ]
    root = Path(__file__).resolve().parent.parent
    env = dict(os.environ, HIP_VISIBLE_DEVICES="", CUDA_VISIBLE_DEVICES="")
    r = subprocess.run(
        [sys.executable, str(root / "bin" / "trace_run"), "--model", path,
         "--dtype", "float32", "--out", str(tmp_path / "o"),
         "--max-tokens", "128"],
        input="".join(json.dumps(s) + "\n" for s in steps), text=True,
        capture_output=True, env=env, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [
        "done 0", "done 1", "done 2"]
    ra, rb = oracle.forward(W, cfg, a)[0], oracle.forward(W, cfg, b)[0]
    V = cfg["vocab"]
    g0 = np.fromfile(tmp_path / "o" / "0.f32", dtype="<f4").reshape(-1, V)
    g2 = np.fromfile(tmp_path / "o" / "2.f32", dtype="<f4").reshape(-1, V)
    assert not (tmp_path / "o" / "1.f32").exists()
    close(g0, ra[[0, 4]], 2e-4)
    close(g2, np.stack([ra[8], rb[3]]), 2e-4)


def test_bench_configurations_are_comparable():
    """The speed comparison runs both models at equal width, head sizes
    and routed experts, and its sizes run through the model."""
    root = Path(__file__).resolve().parent.parent
    sys.path.insert(0, str(root / "tools"))
    try:
        import bench_defosun as bd
    finally:
        sys.path.pop(0)
    for sz in bd.SIZES.values():
        dfo, boz = bd._configs(sz)
        assert dfo.hidden_size == boz.hidden_size == sz["width"]
        assert len(dfo.layer_runs) == boz.num_layers
        a, b = dfo.layers[0].mixer, boz.layers[0].mixer.left
        for k in ("heads", "kv_heads", "dim", "vdim"):
            assert getattr(a, k) == getattr(b, k)
        d, m = dfo.layers[1].mixer, boz.layers[0].mixer.right
        assert (d.heads, d.dim, d.vdim) == (m.heads, m.dim, m.vdim)
        for x, y in zip(dfo.layers, boz.layers):
            for k in ("experts", "top", "expert_ff", "limit"):
                assert getattr(x.mlp, k) == getattr(y.mlp, k)
