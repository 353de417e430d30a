"""Bivatar (post-norm decoder: windowed attention with kept first tokens
and a distance bias / latent attention with borrowed latents, gelu-gated
feed-forward) against a plain float64 model written from the equations
(tests/bivatar_oracle.py).

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

import bivatar_oracle as oracle
from inference_gateway_amd import ops
from inference_gateway_amd.engine.config import (BivatarConfig,
                                                 EngineConfig,
                                                 SamplingParams,
                                                 YarnRotarySpec)
from inference_gateway_amd.engine.engine import LLMEngine
from inference_gateway_amd.engine.models.registry import (
    is_recurrent, model_config_from_dir)

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]


def _dev(device):
    return "cuda:0" if device == "cuda" else "cpu"


def i32(x, device):
    return torch.tensor(x, dtype=torch.int32, device=device)


def f32(x, device):
    return torch.tensor(np.asarray(x), dtype=torch.float32, device=device)


# configurations; sizes all differ from one another
def cfg_small():
    rot = oracle.rot(6, 100.0, 3.0, 16, 4.0, 1.0)
    return oracle.make_config(40, 61, [
        oracle.latent_layer(4, 5, rot, 7, 12, 9, 0.35,
                            mlp=oracle.dense(24)),
        oracle.attention_layer(4, 2, 6, 9, 7, 2, 0.4,
                               mlp=oracle.dense(18)),
        oracle.latent_layer(3, 4, rot, 5, 12, 11, 0.3, kv_from=0),
        oracle.attention_layer(6, 3, 8, 5, 5, 4, 0.3,
                               mlp=oracle.dense(10))], mult=0.4)


def cfg_ones():
    """Single heads and groups, a window of one token, one kept token or
    none, a window longer than any request, no frequency interpolation,
    unit multiplier and embedding scale, layers without feed-forward, one
    rotated pair, latents of one entry."""
    return oracle.make_config(24, 37, [
        oracle.attention_layer(1, 1, 5, 3, 1, 1, 0.45),
        oracle.latent_layer(1, 1, oracle.rot(2, 10.0), 1, 1, 1, 0.6,
                            mlp=oracle.dense(1)),
        oracle.attention_layer(3, 3, 4, 4, 1000, 3, 0.5,
                               mlp=oracle.dense(8)),
        oracle.attention_layer(2, 1, 3, 4, 6, 0, 0.6)],
        scale=1.0, mult=1.0, eps=1e-6)


def cfg_wide():
    """Widths that straddle the kernels' tile sizes: more than 64 value
    entries per head, key and latent widths off the powers of two, many
    heads on one key/value head, kept tokens past one tile, two layers
    on one layer's latents."""
    rot = oracle.rot(20, 1000.0, 8.0, 64, 16.0, 2.0)
    return oracle.make_config(72, 83, [
        oracle.attention_layer(6, 1, 20, 66, 12, 70, 0.22,
                               mlp=oracle.dense(50)),
        oracle.latent_layer(5, 33, rot, 70, 68, 40, 0.15),
        oracle.latent_layer(10, 12, rot, 24, 68, 31, 0.2, kv_from=1,
                            mlp=oracle.dense(33)),
        oracle.latent_layer(2, 30, rot, 9, 68, 17, 0.2, kv_from=1)],
        mult=0.25)


CONFIGS = {"small": cfg_small, "ones": cfg_ones, "wide": cfg_wide}


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


def close(got, ref, tol):
    """Mean-free relative RMS difference per row, like a logit check."""
    got = torch.as_tensor(np.asarray(got.cpu() if torch.is_tensor(got)
                                     else got)).double()
    ref = torch.as_tensor(np.asarray(ref)).double()
    d = got - ref
    d = d - d.mean(-1, keepdim=True)
    err = d.pow(2).mean(-1).sqrt() / ref.pow(2).mean().sqrt()
    assert float(err.max()) < tol, f"rel err {float(err.max()):.3e}"


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
def test_yarn_frequencies_against_the_formula():
    cases = [(12, 500.0, 4.0, 40.0, 8.0, 0.5),   # ramp inside
             (8, 10000.0, 16.0, 4.0, 32.0, 1.0),  # ramp clipped at pair 0
             (4, 10.0, 2.0, 1e6, 2.0, 1.0),       # ramp past the last pair
             (6, 100.0, 1.0, 64.0, 8.0, 1.0)]     # factor 1: plain
    for dims, base, factor, orig, fast, slow in cases:
        f, mag = YarnRotarySpec(base=base, dims=dims, factor=factor,
                                original=orig, fast=fast,
                                slow=slow).frequencies()
        rf, rmag = oracle.rotary_frequencies(oracle.rot(
            dims, base, factor, orig, fast, slow))
        np.testing.assert_allclose(f, rf, rtol=1e-12)
        assert abs(mag - rmag) < 1e-12
    f, mag = YarnRotarySpec(base=500.0, dims=12, factor=4.0, original=40.0,
                            fast=8.0, slow=0.5).frequencies()
    plain = [500.0 ** (-2.0 * i / 12) for i in range(6)]
    # the first pair keeps its frequency, the last is slowed by the
    # factor, something in between is interpolated
    assert f[0] == plain[0] and abs(f[5] - plain[5] / 4.0) < 1e-15
    assert any(plain[i] / 4.0 < f[i] < plain[i] for i in range(1, 5))
    assert abs(mag - (0.1 * np.log(4.0) + 1.0)) < 1e-12


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dims", [(3, 2, 5), (8, 4, 6), (64, 2, 0),
                                  (10, 1, 3)])
def test_half_split_rotation(device, dims):
    """Entry i with entry i + n, scaled cos and sin, only on the slice
    behind `offset`; positions far apart in one batch."""
    n, H, off = dims
    pos = [0, 1, 7, 900, 12345]
    g = torch.Generator().manual_seed(n)
    x = torch.randn(len(pos), H, off + 2 * n + 3, generator=g)
    r = oracle.rot(2 * n, 300.0, 4.0, 32, 8.0, 1.0)
    freq, mag = oracle.rotary_frequencies(r)
    ref = x.double().numpy().copy()
    ref[:, :, off:off + 2 * n] = oracle.rotate_halves(
        ref[:, :, off:off + 2 * n], r, pos)
    y = x.clone().to(device)
    ops.rope_pairs_(y, i32(pos, device), f32(freq, device), off, True, mag)
    # fp32 angles: 12345 rad carries 5e-4
    np.testing.assert_allclose(y.cpu().numpy(), ref, atol=4e-3)
    np.testing.assert_allclose(y.cpu().numpy()[:4], ref[:4], atol=2e-4)
    # the interleaved layout pairs other entries
    z = ops.rope_pairs_(x.clone().to(device), i32(pos, device),
                        f32(freq, device), off, False, mag)
    if n > 1:
        assert np.abs(z.cpu().numpy()[1:] - ref[1:]).max() > 1e-2


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dims", [(9, 12, 6, 4), (1, 1, 2, 1),
                                  (300, 270, 64, 20)])
def test_latent_rows_of_a_projection(device, dims):
    """Both norms, the rotated key, the gates and the paged rows; and the
    form of a layer without keys of its own."""
    Q, R, E, H = dims
    pos = [5, 6, 0, 1, 77]
    T, bs = len(pos), 4
    g = torch.Generator().manual_seed(Q)
    down = torch.randn(T, Q + R + E + H, generator=g) * 2
    qw, kw = torch.randn(Q, generator=g), torch.randn(R, generator=g)
    r = oracle.rot(E, 50.0, 2.0, 16, 4.0, 1.0)
    freq, mag = oracle.rotary_frequencies(r)
    x = down.double().numpy()
    q_ref = oracle.rms_unit(x[:, :Q], 1e-5) * qw.double().numpy()
    rows_ref = np.concatenate([
        oracle.rms_unit(x[:, Q:Q + R], 1e-5) * kw.double().numpy(),
        oracle.rotate_halves(x[:, None, Q + R:Q + R + E], r, pos)[:, 0]],
        -1)
    g_ref = oracle.sigmoid(x[:, Q + R + E:])
    slots = [2 * bs + 1, 2 * bs + 2, 5 * bs, 5 * bs + 1, 3]
    cache = torch.zeros(6, bs, R + E, device=device)
    cq, gate = ops.latent_down_post(
        down.to(device), i32(pos, device), i32(slots, device), cache,
        qw.to(device), kw.to(device), f32(freq, device), 1e-5, Q, R, E, H,
        True, mag)
    np.testing.assert_allclose(cq.cpu().numpy(), q_ref, atol=3e-5,
                               rtol=3e-5)
    np.testing.assert_allclose(gate.cpu().numpy(), g_ref, atol=1e-6)
    flat = cache.view(-1, R + E).cpu().numpy()
    np.testing.assert_allclose(flat[slots], rows_ref, atol=6e-5, rtol=3e-5)
    assert not np.delete(flat, slots, 0).any()
    own = torch.cat([down[:, :Q], down[:, Q + R + E:]], 1).to(device)
    cq2, gate2 = ops.latent_down_post(
        own, i32(pos, device), i32(slots, device), None, qw.to(device), None,
        f32(freq, device), 1e-5, Q, R, E, H, True, mag)
    np.testing.assert_allclose(cq2.cpu().numpy(), q_ref, atol=3e-5,
                               rtol=3e-5)
    np.testing.assert_allclose(gate2.cpu().numpy(), g_ref, atol=1e-6)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("width", [8, 7, 130])
def test_gelu_gated_activation(device, width):
    g = torch.Generator().manual_seed(width)
    x = torch.randn(5, 2 * width, generator=g) * 4
    x[0, 0], x[0, 1] = 30.0, -30.0
    z = x.double().numpy()
    ref = oracle.gelu_tanh(z[:, :width]) * z[:, width:]
    out = ops.gated_act(x.to(device), ops.GATED_ACT_GELU)
    np.testing.assert_allclose(out.cpu().numpy(), ref, atol=5e-6, rtol=2e-5)
    out = ops.gated_act(x.bfloat16().to(device), ops.GATED_ACT_GELU)
    np.testing.assert_allclose(out.float().cpu().numpy(), ref, atol=0.1,
                               rtol=3e-2)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("D", [50, 256, 704, 5000])
def test_scaled_post_norm_update(device, D):
    """residual += m * rms(delta) * w and the copy the next product
    reads; then the same with a norm of the sum (the model's last)."""
    g = torch.Generator().manual_seed(D)
    res = torch.randn(5, D, generator=g) * 3
    delta = torch.randn(5, D, generator=g) * 7
    w, wf = torch.randn(D, generator=g), torch.randn(D, generator=g)
    ref = res.double().numpy() + 0.3 * oracle.rms_unit(
        delta.double().numpy(), 1e-5) * w.double().numpy()
    x = res.clone().to(device)
    out = ops.add_normed_rmsnorm(x, delta.to(device), w.to(device), None,
                                 1e-5, torch.float32, 0.3)
    np.testing.assert_allclose(x.cpu().numpy(), ref, atol=2e-5, rtol=2e-5)
    np.testing.assert_array_equal(out.cpu().numpy(), x.cpu().numpy())
    x = res.clone().to(device)
    out = ops.add_normed_rmsnorm(x, delta.to(device), w.to(device),
                                 wf.to(device), 1e-5, torch.float32, 0.3)
    np.testing.assert_allclose(
        out.cpu().numpy(), oracle.rms_unit(ref, 1e-5) * wf.double().numpy(),
        atol=3e-5, rtol=3e-5)
    # bfloat16 sublayer output and copy around the fp32 stream
    d16 = delta.bfloat16()
    ref16 = res.double().numpy() + 0.3 * oracle.rms_unit(
        d16.double().numpy(), 1e-5) * w.double().numpy()
    x = res.clone().to(device)
    out = ops.add_normed_rmsnorm(x, d16.to(device), w.to(device), None, 1e-5,
                                 torch.bfloat16, 0.3)
    np.testing.assert_allclose(x.cpu().numpy(), ref16, atol=2e-5, rtol=2e-5)
    torch.testing.assert_close(out.cpu(), x.cpu().bfloat16())
    # nothing to add: the plain cast
    x = res.clone().to(device)
    out = ops.add_normed_rmsnorm(x, None, None, None, 1e-5, torch.bfloat16,
                                 0.3)
    torch.testing.assert_close(out.cpu(), res.bfloat16())


class WindowCase:
    """One sequence's keys and values in scattered pages."""

    def __init__(self, device, dtype, H, G, N, P, bs, ctx, seed=0):
        g = torch.Generator().manual_seed(ctx + N + seed)
        self.device, self.dtype = device, dtype
        self.H, self.G, self.N, self.P, self.bs = H, G, N, P, bs
        self.q = torch.randn(ctx, H, N, generator=g)
        self.k = torch.randn(ctx, G, N, generator=g)
        self.v = torch.randn(ctx, G, P, generator=g)
        self.gate = torch.randn(ctx, H + 3, generator=g)
        nb = (ctx + bs - 1) // bs
        self.perm = torch.randperm(nb + 3, generator=g)[:nb].tolist()
        self.nb = nb

    def match(self, qi, kj, length):
        """Query qi and key kj get one direction and `length`."""
        self.k[kj] = self.k[kj] / self.k[kj].norm(dim=-1, keepdim=True) \
            * length
        self.q[qi] = self.k[kj].repeat_interleave(self.H // self.G, 0)

    def reference(self, scale, window, keep, slopes=True, gate=True,
                  rows=None):
        q, k, v, gt = (x.to(self.dtype).double().numpy()
                       for x in (self.q, self.k, self.v, self.gate))
        o = oracle.window_attention(
            q, k, v, self.H, self.G, scale, window, keep,
            None if slopes else [0.0] * self.H, rows)
        if gate:
            gt = gt if rows is None else gt[rows]
            o = o * oracle.sigmoid(gt[:, :self.H])[:, :, None]
        return o

    def run(self, scale, window, keep, rows=None, slopes=True, gate=True,
            portion=False):
        """rows None: the whole sequence as a prompt; else each listed
        position as a decoded row of its own sequence entry, or with
        `portion` the (consecutive) positions as one prompt portion."""
        dev, dt, ctx = self.device, self.dtype, self.q.shape[0]
        kc = torch.zeros(self.nb + 3, self.G, self.bs, self.N, dtype=dt,
                         device=dev)
        vc = torch.zeros(self.nb + 3, self.G, self.bs, self.P, dtype=dt,
                         device=dev)
        slots = [self.perm[j // self.bs] * self.bs + j % self.bs
                 for j in range(ctx)]
        ops.append_paged_kv(self.k.reshape(ctx, -1).to(dt).to(dev),
                            self.v.reshape(ctx, -1).to(dt).to(dev), kc, vc,
                            i32(slots, dev))
        extra = dict(keep=keep)
        if slopes:
            extra["slopes"] = f32(oracle.distance_slopes(self.H), dev)
        sel = list(range(ctx)) if rows is None else rows
        n = len(sel)
        if gate:
            extra["gate"] = self.gate.to(dt).to(dev)[sel][:, :self.H]
        q = self.q.reshape(ctx, -1).to(dt).to(dev)[sel]
        if rows is None or portion:
            out = ops.softcap_attention(
                q, kc, vc, i32([self.perm], dev), i32([0] * n, dev),
                i32(sel, dev), scale, 0.0, 0.0, 1, window, n, [n],
                i32([0, n], dev), i32([sel[0]], dev), **extra)
        else:
            out = ops.softcap_attention(
                q, kc, vc, i32([self.perm] * n, dev),
                i32(list(range(n)), dev), i32(sel, dev), scale, 0.0, 0.0, 1,
                window, 0, None, i32(list(range(n + 1)), dev),
                i32(sel, dev), **extra)
        return out.float().cpu().numpy().reshape(n, self.H, self.P)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dims", [
    # H, G, N, P, page, window, keep
    (4, 2, 6, 9, 4, 7, 3), (1, 1, 5, 3, 2, 1, 1), (6, 1, 20, 66, 8, 30, 2),
    (2, 2, 64, 64, 16, 64, 5), (8, 4, 16, 8, 4, 0, 4),
    (3, 3, 8, 1, 4, 5, 0), (2, 1, 4, 4, 4, 9, 40)])
def test_window_attention_alone(device, dims):
    H, G, N, P, bs, window, keep = dims
    c = WindowCase(device, torch.float32, H, G, N, P, bs, 75)
    ref = c.reference(0.4, window, keep)
    np.testing.assert_allclose(c.run(0.4, window, keep), ref, atol=3e-5,
                               rtol=3e-5)
    rows = [0, 1, keep, 6, 7, 8, 31, 32, 74]
    np.testing.assert_allclose(c.run(0.4, window, keep, rows), ref[rows],
                               atol=3e-5, rtol=3e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("window,keep", [(16, 3), (33, 8), (64, 64), (5, 1)])
def test_window_and_kept_edges(device, window, keep):
    """One key stands out for one query.  Just inside the window and
    among the kept tokens it owns the output; one token further out it
    leaves no trace at all; in a prompt and decoded."""
    ctx = 3 * window + keep + 7
    qi = ctx - 3
    spots = {qi - window + 1: True, qi - window: False, keep - 1: True,
             keep: qi - keep < window, 0: True}
    for kj, seen in spots.items():
        c = WindowCase(device, torch.float32, 2, 1, 8, 4, 4, ctx)
        c.match(qi, kj, 12.0)
        near = [qi - 1, qi, qi + 1]
        ref = c.reference(1.0, window, keep, slopes=False, gate=False,
                          rows=near)
        mine = np.abs(ref[1] - c.v[kj].numpy()).max() < 1e-3
        assert mine == seen, (kj, seen)
        one = c.run(1.0, window, keep, near, slopes=False, gate=False)
        np.testing.assert_allclose(one, ref, atol=3e-5, rtol=3e-5)
        part = c.run(1.0, window, keep, near, slopes=False, gate=False,
                     portion=True)
        np.testing.assert_allclose(part, ref, atol=3e-5, rtol=3e-5)
        if not seen:
            # moving the unseen key changes nothing
            c.k[kj] *= -1.0
            again = c.run(1.0, window, keep, [qi], slopes=False, gate=False)
            np.testing.assert_array_equal(again, one[1:2])


@pytest.mark.parametrize("device", DEVICES)
def test_kept_key_keeps_its_distance(device):
    """A kept first token 280 positions back is penalised by its true
    distance, not by its place among the visible keys: the head with the
    small slope still finds it, the head with the large one does not."""
    c = WindowCase(device, torch.float32, 2, 1, 8, 5, 16, 300)
    v = c.v[4, 0].numpy()
    rows = [284, 285, 286]
    for length, found in ((8.0, True), (3.0, False)):
        # score 64, then 9; slopes 1/16 and 1/256 take 17.6 and 1.1 off
        c.match(285, 4, length)
        ref = c.reference(1.0, 20, 6, gate=False, rows=rows)
        assert (np.abs(ref[1, 0] - v).max() < 1e-3) == found
        if found:
            assert np.abs(ref[1, 1] - v).max() < 1e-3
        for portion in (False, True):
            out = c.run(1.0, 20, 6, rows, gate=False, portion=portion)
            np.testing.assert_allclose(out, ref, atol=3e-5, rtol=3e-5)


@pytest.mark.gpu
@pytest.mark.parametrize("dims", [
    # H, G, N, P, page, window, keep
    (4, 2, 64, 64, 16, 48, 5), (9, 3, 88, 176, 16, 100, 70),
    (8, 2, 128, 128, 8, 0, 0), (3, 1, 24, 72, 4, 70, 1),
    (16, 1, 128, 64, 16, 33, 130), (6, 6, 48, 40, 16, 1, 64)])
def test_window_tile_kernel_bf16(dims):
    """The MFMA path over its padded instantiations: a prompt of several
    tiles, kept tiles ahead of the window's, decoded rows."""
    H, G, N, P, bs, window, keep = dims
    c = WindowCase("cuda:0", torch.bfloat16, H, G, N, P, bs, 230)
    ref = c.reference(N ** -0.5, window, keep)
    assert np.abs(c.run(N ** -0.5, window, keep) - ref).max() < 0.06
    rows = [0, 3, 63, 64, 65, 128, 200, 229]
    out = c.run(N ** -0.5, window, keep, rows)
    assert np.abs(out - ref[rows]).max() < 0.06
    if window and keep:
        # a kept key far behind the window, and the first key not kept
        for kj in (0, keep - 1, min(keep, 228)):
            c.match(229, kj, N ** 0.5 * 2.0)
            ref = c.reference(N ** -0.5, window, keep)
            out = c.run(N ** -0.5, window, keep)
            assert np.abs(out - ref).max() < 0.06
            one = c.run(N ** -0.5, window, keep, [229])
            assert np.abs(one - ref[229:]).max() < 0.06


class LatentCase:
    """Queries of one sequence against latent rows in scattered pages."""

    def __init__(self, device, dtype, H, N, R, E, P, bs, ctx, seed=0):
        g = torch.Generator().manual_seed(ctx + R + seed)
        self.device, self.dtype, self.bs = device, dtype, bs
        self.H, self.N, self.R, self.E, self.P = H, N, R, E, P
        rnd = lambda *s: torch.randn(*s, generator=g).to(dtype)  # noqa: E731
        self.q = rnd(ctx, H, N + E)
        self.c, self.kr = rnd(ctx, R), rnd(ctx, E)
        self.uk = (rnd(H, N, R).float() * R ** -0.5).to(dtype)
        self.uv = (rnd(H, P, R).float() * R ** -0.5).to(dtype)
        self.gate = torch.rand(ctx, H, generator=g)
        nb = (ctx + bs - 1) // bs
        self.perm = torch.randperm(nb + 2, generator=g)[:nb].tolist()
        self.nb = nb

    def reference(self, scale):
        q, c, kr, uk, uv, gt = (x.double().numpy() for x in (
            self.q, self.c, self.kr, self.uk, self.uv, self.gate))
        T = len(c)
        kn = np.stack([c @ uk[h].T for h in range(self.H)], 1)
        v = np.stack([c @ uv[h].T for h in range(self.H)], 1)
        return oracle.latent_attention(q, kn, kr, v, self.N, scale) \
            * gt[:, :, None]

    def run(self, scale, rows=None):
        dev, dt, ctx = self.device, self.dtype, len(self.c)
        cache = torch.zeros(self.nb + 2, self.bs, self.R + self.E, dtype=dt,
                            device=dev)
        slots = [self.perm[j // self.bs] * self.bs + j % self.bs
                 for j in range(ctx)]
        cache.view(-1, self.R + self.E)[slots] = torch.cat(
            [self.c, self.kr], 1).to(dev)
        sel = list(range(ctx)) if rows is None else rows
        n = len(sel)
        q = self.q[sel].to(dev)
        qa = torch.stack([q[:, h, :self.N] @ self.uk[h].to(dev)
                          for h in range(self.H)], 1)
        if rows is None:
            o = ops.latent_attention(
                qa, q[:, :, self.N:], cache, i32([self.perm], dev),
                i32([0] * n, dev), i32(sel, dev), None, scale, 0, n, [n],
                ctx, self.gate[sel].to(dev))
        else:
            o = ops.latent_attention(
                qa, q[:, :, self.N:], cache, i32([self.perm] * n, dev),
                i32(list(range(n)), dev), i32(sel, dev), None, scale, 0, 0,
                None, ctx, self.gate[sel].to(dev))
        return torch.stack([o[:, h].float() @ self.uv[h].float().to(dev).t()
                            for h in range(self.H)], 1).cpu().numpy()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dims", [(4, 5, 12, 6, 7, 4), (1, 1, 1, 2, 1, 2),
                                  (5, 33, 68, 20, 70, 8),
                                  (3, 16, 64, 16, 24, 16)])
def test_latent_attention_alone(device, dims):
    """No sink, no window, one gate per head; the absorbed form against
    per-head keys and values; a far key that stands out for one query."""
    H, N, R, E, P, bs = dims
    c = LatentCase(device, torch.float32, H, N, R, E, P, bs, 75)
    # the shared rotated part carries the outlier
    c.kr[3] = c.kr[3] / c.kr[3].norm() * 6.0
    c.q[70, :, N:] = c.kr[3]
    ref = c.reference(0.3)
    np.testing.assert_allclose(c.run(0.3), ref, atol=5e-5, rtol=5e-5)
    rows = [0, 1, 8, 31, 32, 70, 74]
    np.testing.assert_allclose(c.run(0.3, rows), ref[rows], atol=5e-5,
                               rtol=5e-5)


@pytest.mark.gpu
@pytest.mark.parametrize("dims", [
    # H, N, latent, rotated, value, page
    (8, 64, 64, 16, 48, 16), (12, 40, 96, 32, 40, 16), (3, 24, 72, 12, 20, 4),
    (20, 32, 256, 64, 32, 16), (40, 16, 136, 24, 8, 8), (1, 8, 10, 6, 4, 16),
    (70, 8, 32, 8, 8, 16)])
def test_latent_tile_kernel_bf16(dims):
    """The MFMA path without sinks and with the gate fused in: prompts of
    several tiles, decoded rows with and without key splits."""
    H, N, R, E, P, bs = dims
    c = LatentCase("cuda:0", torch.bfloat16, H, N, R, E, P, bs, 330)
    scale = (N + E) ** -0.5
    c.kr[3] = (c.kr[3].float() / c.kr[3].float().norm() * E ** 0.5
               * 3.0).to(torch.bfloat16)
    c.q[320, :, N:] = c.kr[3]
    ref = c.reference(scale)
    assert np.abs(c.run(scale) - ref).max() < 0.08
    rows = [0, 1, 31, 32, 33, 200, 320, 329]
    assert np.abs(c.run(scale, rows) - ref[rows]).max() < 0.08
    many = [(7 * i) % 330 for i in range(300)]
    assert np.abs(c.run(scale, many) - ref[many]).max() < 0.08


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
    eng.model.tap = lambda i, x: taps.append(x.double().cpu().numpy())
    got = replay_all(eng, t, [41])
    eng.model.tap = None
    assert len(taps) == len(cfg["layers"])
    for i, (a, b) in enumerate(zip(taps, taps_ref)):
        assert np.abs(a - b).max() < 2e-4 * max(1.0, np.abs(b).max()), i
    close(got, ref, 2e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_portions_and_token_by_token(tmp_path, device, name):
    """The same request whole, token by token, and in ragged portions
    down to two tokens (cut inside pages and windows); pages are reused
    from run to run."""
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
def test_first_tokens_in_used_pages(tmp_path, device):
    """Requests of one, two and three tokens in pages that longer
    requests have just left: nothing of the old keys and latents shows."""
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
def test_long_decode(tmp_path, device):
    """Windows pass over decoded tokens many times; kept first tokens
    stay in sight to the end."""
    cfg = cfg_small()
    W = oracle.random_weights(cfg, 16)
    eng = make_engine(tmp_path, cfg, W, device, blocks=80)
    t = toks(260, cfg["vocab"], 17)
    ref, _ = oracle.forward(W, cfg, t)
    close(replay_all(eng, t, [6] + [1] * 254), ref, 3e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_kept_tokens_reach_the_logits(tmp_path, device):
    """Weights that make a kept first token decisive for a far query:
    the engine follows the oracle, and the oracle moves when the kept
    token is no longer kept."""
    cfg = oracle.make_config(32, 41, [
        oracle.attention_layer(2, 1, 8, 8, 6, 3, 4.0)], mult=1.0)
    W = oracle.random_weights(cfg, 71)
    # token 9's query meets token 7's key head on
    W["embed"][7], W["embed"][9] = 0.0, 0.0
    W["embed"][7, 0] = W["embed"][9, 1] = 1.0
    W["l0.mix.k"][:, 0] = W["l0.mix.q"][:, 1] = 0.0
    W["l0.mix.k"][0, 0] = W["l0.mix.q"][0, 1] = W["l0.mix.q"][8, 1] = 1.0
    t = [x if x not in (7, 9) else 8 for x in toks(90, 41, 72)]
    t[2], t[60], t[89] = 7, 9, 9               # token 2 is the last kept
    ref, _ = oracle.forward(W, cfg, t)
    other = json.loads(json.dumps(cfg))
    other["layers"][0]["mixer"]["mask"]["keep_first"] = 2
    moved = np.abs(oracle.forward(W, other, t)[0] - ref)
    assert moved[89].max() > 1e-2 and moved[:8].max() < 1e-12
    eng = make_engine(tmp_path, cfg, W, device)
    close(replay_all(eng, t, [90]), ref, 2e-4)
    close(replay_all(eng, t, [50, 2, 7] + [1] * 31), ref, 2e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_borrowed_latents_follow_the_source_layer(tmp_path, device):
    """The borrowing layers read the rows their source layer wrote in
    the SAME step, also when the request arrives in portions; changing
    the source's latents changes the borrowers' output too, and a
    borrower keeps nothing of its own."""
    cfg = cfg_wide()
    W = oracle.random_weights(cfg, 31)
    t = toks(45, cfg["vocab"], 32)
    eng = make_engine(tmp_path / "a", cfg, W, device)
    assert eng.kv_caches[2] == () and eng.kv_caches[3] == ()
    ref, _ = oracle.forward(W, cfg, t)
    close(replay_all(eng, t, [20, 1, 1, 23]), ref, 2e-4)
    W2 = dict(W)
    W2["l1.mix.dkv"] = -W["l1.mix.dkv"]
    ref2, _ = oracle.forward(W2, cfg, t)
    assert np.abs(ref2 - ref).max() > 1e-3
    eng2 = make_engine(tmp_path / "b", cfg, W2, device)
    close(replay_all(eng2, t, [45]), ref2, 2e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_bfloat16_mode(tmp_path, device):
    cfg = cfg_small()
    W = oracle.random_weights(cfg, 18)
    eng = make_engine(tmp_path, cfg, W, device, dtype="bfloat16")
    t = toks(33, cfg["vocab"], 19)
    ref, _ = oracle.forward(W, cfg, t)
    close(replay_all(eng, t, [33]), ref, 6e-2)
    close(replay_all(eng, t, [5, 2, 1, 1, 20, 4]), ref, 6e-2)


@pytest.mark.gpu
def test_bfloat16_tile_sizes_through_the_engine(tmp_path):
    """Head and latent sizes that take the MFMA attention paths, a
    prompt of several tiles, portions and decoded rows, in bfloat16."""
    rot = oracle.rot(24, 10000.0, 4.0, 64, 32.0, 1.0)
    cfg = oracle.make_config(128, 97, [
        oracle.attention_layer(6, 2, 32, 24, 50, 9, 0.18,
                               mlp=oracle.dense(200)),
        oracle.latent_layer(6, 40, rot, 32, 88, 64, 0.125,
                            mlp=oracle.dense(160)),
        oracle.latent_layer(4, 32, rot, 40, 88, 72, 0.13, kv_from=1,
                            mlp=oracle.dense(120))], mult=0.5)
    W = oracle.random_weights(cfg, 51)
    eng = make_engine(tmp_path, cfg, W, "cuda", dtype="bfloat16", blocks=40,
                      block=16)
    t = toks(200, cfg["vocab"], 52)
    ref, _ = oracle.forward(W, cfg, t)
    close(replay_all(eng, t, [200]), ref, 6e-2)
    close(replay_all(eng, t, [70, 2, 100, 1, 1, 26]), ref, 6e-2)


def _greedy(cfg, W, prompt, n):
    t = list(prompt)
    for _ in range(n):
        t.append(int(np.argmax(oracle.forward(W, cfg, t)[0][-1])))
    return t[len(prompt):]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("mode", ["plain", "chunked_mixed", "prefix"])
def test_greedy_generation_through_scheduler(tmp_path, device, mode):
    """Everything the model keeps is paged, so prefix caching serves it
    too: the second request of a prompt starts behind its cached pages."""
    cfg = cfg_small()
    W = oracle.random_weights(cfg, 21)
    kw = {}
    if mode == "chunked_mixed":
        kw = dict(enable_chunked_prefill=True, enable_mixed_batches=True,
                  max_batched_tokens=7)
    elif mode == "prefix":
        kw = dict(enable_prefix_caching=True)
    eng = make_engine(tmp_path, cfg, W, device, **kw)
    prompts = [toks(n, cfg["vocab"], 30 + n) for n in (5, 19, 11)]
    if mode == "prefix":
        prompts.append(prompts[1][:17] + prompts[2][:3])
    sp = SamplingParams(max_new_tokens=6, temperature=0.0)
    rids = []
    for wave in (prompts[:3], prompts[3:]):
        rids += [eng.add_request(p, sp) for p in wave]
        for _ in range(200):
            if eng.is_finished():
                break
            eng.step()
    for rid, p in zip(rids, prompts):
        assert eng.get_output(rid).token_ids == _greedy(cfg, W, p, 6)


@pytest.mark.parametrize("device", DEVICES)
def test_preemption_resumes(tmp_path, device):
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
def test_forked_group_copies_the_tail_page(tmp_path, device):
    """n=2 from one prefill: the branch shares the prompt's full pages
    and gets a copy of the partial one, keys, values and latents."""
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
    cfg = cfg_wide()
    W = oracle.random_weights(cfg, 22)
    path = oracle.save_checkpoint(tmp_path / "m", cfg, W)
    mc = model_config_from_dir(path)
    assert isinstance(mc, BivatarConfig) and not is_recurrent(mc)
    assert [l.type for l in mc.layers] == ["attention"] \
        + ["latent_attention"] * 3
    assert mc.layers[2].mixer.kv_from == 1 and mc.layers[1].mlp is None
    assert (mc.layers[0].mixer.window, mc.layers[0].mixer.keep_first) == (
        12, 70)
    assert mc.layers[1].mixer.rot.factor == 8.0 and mc.residual_mult == 0.25
    # only the layers that own keys page anything
    assert mc.kv_bytes_per_token(2) == 2 * ((20 + 66) + (68 + 20))
    # the query latent's size comes from the tensors when the json has none
    bare = json.loads(json.dumps(cfg))
    for l in bare["layers"][1:]:
        del l["mixer"]["q_rank"]
    p2 = oracle.save_checkpoint(tmp_path / "m2", bare, W)
    assert model_config_from_dir(p2).layers[2].mixer.q_rank == 31
    bad = dict(W)
    bad["l1.mix.dkv"] = bad["l1.mix.dkv"][:-1]
    with pytest.raises(ValueError, match="l1.mix.dq"):
        make_engine(tmp_path / "e", cfg, bad, "cpu")
    unknown = oracle.make_config(8, 9, [{"type": "lstm", "mixer": {},
                                         "mlp": None}])
    with pytest.raises(ValueError, match="unknown mixer"):
        BivatarConfig.from_dict(unknown)
    with pytest.raises(ValueError, match="unknown mlp"):
        BivatarConfig.from_dict(oracle.make_config(8, 9, [
            oracle.attention_layer(1, 1, 4, 4, 8, 1, 0.5,
                                   mlp={"kind": "moe"})]))
    rot = oracle.rot(2, 10.0)
    for layers in (
            [oracle.latent_layer(1, 2, rot, 2, 4, 4, 0.5, kv_from=1),
             oracle.latent_layer(1, 2, rot, 2, 4, 4, 0.5)],
            [oracle.attention_layer(1, 1, 4, 4, 8, 1, 0.5),
             oracle.latent_layer(1, 2, rot, 2, 4, 4, 0.5, kv_from=0)],
            [oracle.latent_layer(1, 2, rot, 2, 4, 4, 0.5),
             oracle.latent_layer(1, 2, rot, 2, 4, 4, 0.5, kv_from=0),
             oracle.latent_layer(1, 2, rot, 2, 4, 4, 0.5, kv_from=1)]):
        with pytest.raises(ValueError, match="kv_from"):
            BivatarConfig.from_dict(oracle.make_config(8, 9, layers))
    with pytest.raises(ValueError, match="differs"):
        BivatarConfig.from_dict(oracle.make_config(8, 9, [
            oracle.latent_layer(1, 2, rot, 2, 4, 4, 0.5),
            oracle.latent_layer(1, 2, rot, 2, 6, 4, 0.5, kv_from=0)]))


def test_preset_runs(tmp_path):
    eng = LLMEngine(EngineConfig.tiny_bivatar(), device="cpu")
    rid = eng.add_request(list(range(1, 20)),
                          SamplingParams(max_new_tokens=4, temperature=0.0))
    while not eng.is_finished():
        eng.step()
    assert len(eng.get_output(rid).token_ids) == 4
    assert eng.kv_caches[3] == ()


def test_local_provider_serves_a_checkpoint_directory(tmp_path):
    """The gateway's local provider with LOCAL_MODEL=hf picks the
    architecture from the directory's config.json and generates through
    the async engine with sampling."""
    import asyncio

    from inference_gateway_amd.config import LocalConfig
    from inference_gateway_amd.providers.local import LocalProvider

    cfg = oracle.make_config(48, 300, [
        oracle.attention_layer(2, 1, 8, 10, 12, 2, 0.35,
                               mlp=oracle.dense(32)),
        oracle.latent_layer(2, 8, oracle.rot(4, 100.0), 10, 16, 12, 0.3)])
    W = oracle.random_weights(cfg, 35)
    path = oracle.save_checkpoint(tmp_path / "m", cfg, W)
    lc = LocalConfig(enabled=True, model="hf", max_num_seqs=4,
                     max_model_len=128)
    lc.num_gpu_blocks = 64
    lc.weights_path = path
    provider = LocalProvider(lc, device="cpu")
    try:
        assert isinstance(provider.engine.engine.cfg.model, BivatarConfig)

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
    cfg = cfg_ones()
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
    """The speed comparison runs both models at equal width, head and
    latent sizes and feed-forward parameters."""
    root = Path(__file__).resolve().parent.parent
    sys.path.insert(0, str(root / "tools"))
    try:
        import bench_bivatar as bb
    finally:
        sys.path.pop(0)
    for sz in bb.SIZES.values():
        biv, fed = bb._configs(sz)
        assert biv.hidden_size == fed.hidden_size == sz["width"]
        assert biv.num_layers == fed.num_layers
        assert 3 * biv.layers[0].mlp.ff == 2 * fed.layers[0].mlp.ff
        a, f = biv.layers[1].mixer, fed.layers[1].mixer
        for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank",
                  "window"):
            assert getattr(a, k) == getattr(f, k)
        assert biv.layers[3].mixer.kv_from == 1
