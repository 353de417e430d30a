"""Defosun: a per-layer decoder with several residual streams for the
MI355X engine.

Instead of one residual sum the model carries B fp32 streams, all equal to
the token row at the start.  A sublayer reads one combination of them and
writes into all of them,

    y = f(norm(sum_b a_b X_b));   X_t <- sum_b M[b, t] X_b + c_t y

with learned a, c [B] and M [B, B] per sublayer; the norm is RMS with a
weight stored around zero, and the streams are summed before the last one.
A run of neighbouring layers may repeat: every pass uses the same weights
and has a cache of its own.  Mixers, chosen per layer:

  SinkRotaryAttention  (engine/models/bozolorn.py) projection biases,
                       half-split partial rotary positions, learned sinks,
                       values that are the keys before rotation
  LatentAttention      (engine/models/fedatar.py) direct queries,
                       interleaved rotary positions, learned sinks
  FixedDecayAttention  linear attention with one fixed decay per head

Feed-forwards: GatedMLP (engine/models/bivatar.py, silu), SharedExpertMoE
or none.  The step between two sublayers is one kernel (ops.stream_step).
"""
from __future__ import annotations

from typing import List

import torch
import torch.nn as nn
import torch.nn.functional as F

from ... import ops
from ...parallel.comm import tp_world_size
from ..config import (DefosunConfig, FixedDecaySpec, SharedClampedMoESpec,
                      SiluFFSpec)
from . import moe_common
from .batch import ForwardBatch
from .bivatar import GatedMLP
from .bozolorn import SinkRotaryAttention, _norm_w, _w
from .fedatar import LatentAttention, _param, _rand


class FixedDecayAttention(nn.Module):
    """q, k, v = silu(W h); per head S <- decay_h S + k v^T, o = S^T q;
    the concatenated heads RMS-normed together, times a weight and
    sigmoid(W_g h), then W_o.  The memory is an fp32 slot buffer; silu is
    applied where the recurrence reads the fused projection."""

    def __init__(self, hidden: int, spec: FixedDecaySpec, eps: float,
                 name: str, device, dtype):
        super().__init__()
        self.spec, self.eps, self.dtype = spec, eps, dtype
        H, N, P = spec.heads, spec.dim, spec.vdim
        # fused projection rows: q | k | v | output-gate logits
        self.qkvg = _w((2 * H * (N + P), hidden), device, dtype,
                       name + ".qkvg", hidden)
        self.norm_w = _norm_w(H * P, device, name + ".norm")
        self.o = _w((hidden, H * P), device, dtype, name + ".o", H * P)
        self.register_buffer("decay", torch.tensor(
            spec.decay, dtype=torch.float32, device=device),
            persistent=False)

    def cache_spec(self) -> tuple:
        s = self.spec
        return ("state", s.heads * s.dim * s.vdim)

    def forward(self, h: torch.Tensor, fb: ForwardBatch, mem: torch.Tensor):
        s = self.spec
        H, N, P = s.heads, s.dim, s.vdim
        T, k0, v0 = h.shape[0], H * N, 2 * H * N
        g0 = v0 + H * P
        proj = F.linear(h, self.qkvg)
        o = ops.fixed_decay_scan(
            proj[:, :k0].view(T, H, N), proj[:, k0:v0].view(T, H, N),
            proj[:, v0:g0].view(T, H, P), self.decay, mem, fb.seq_cu,
            fb.seq_start, fb.seq_slots, fb.seq_rows, True)
        y = ops.head_norm_gate(o, proj[:, g0:], self.norm_w, self.eps, H * P,
                               ops.GATE_SIGMOID, False, None, None,
                               self.dtype)
        return F.linear(y, self.o)


class SharedExpertMoE(nn.Module):
    """Experts are the largest entries of softmax(W_r h) over all experts
    (fp32) and are weighted by those entries.  Expert: W_down (g' sigmoid(
    ALPHA g') (u' + 1)), g' = min(W_gate h, L), u' = clamp(W_up h, -L, L).
    An optional shared expert of the same form (own size and limit) runs
    for every token, times sigmoid(w_sg . h); its gate is one more row of
    the router GEMM.  Expert weights are stored K-major ([E, in, out]),
    gate and up stacked."""

    ALPHA = 1.702
    PADDED_MAX_ROWS = 256

    def __init__(self, hidden: int, spec: SharedClampedMoESpec, name: str,
                 device, dtype):
        super().__init__()
        self.spec = spec
        E, f, sf = spec.experts, spec.expert_ff, spec.shared_ff
        # fp32 rows: router | shared expert's gate
        self.router_w = _w((E + (1 if sf else 0), hidden), device,
                           torch.float32, name + ".router", hidden)
        self.up_t = _w((E, hidden, 2 * f), device, dtype, name + ".up",
                       hidden)
        self.down_t = _w((E, f, hidden), device, dtype, name + ".down", f)
        self.shared_up = self.shared_down = None
        if sf:
            self.shared_up = _w((2 * sf, hidden), device, dtype,
                                name + ".shared.up", hidden)
            self.shared_down = _w((hidden, sf), device, dtype,
                                  name + ".shared.down", sf)

    def _act(self, z: torch.Tensor) -> torch.Tensor:
        return ops.gated_act(z, ops.GATED_ACT_CLAMPED, self.spec.limit,
                             self.ALPHA)

    def forward(self, h: torch.Tensor, fb: ForwardBatch) -> torch.Tensor:
        sp = self.spec
        T, E = h.shape[0], sp.experts
        logits = F.linear(h.float(), self.router_w)
        padded = T <= self.PADDED_MAX_ROWS
        C = (T + 63) // 64 * 64
        weights, idx, dst = ops.moe_topk_route(
            logits[:, :E], sp.top, C if padded else 0, over_all=True)
        if padded and dst is None:
            dst = moe_common.padded_rows(idx, E, C)
        shared = gate = None
        if self.shared_up is not None:
            shared = F.linear(ops.gated_act(
                F.linear(h, self.shared_up), ops.GATED_ACT_CLAMPED,
                sp.shared_limit, self.ALPHA), self.shared_down)
            gate = logits[:, E]
        return moe_common.experts_combined(
            h, weights, idx, dst, C, self.up_t, self.down_t, self._act,
            shared, gate)


class StreamMix(nn.Module):
    """One sublayer's stream weights, fp32: a (read), c (write), M
    ([from, to])."""

    def __init__(self, streams: int, name: str, device):
        super().__init__()
        B = streams
        self.inw = _param(1.0 / B + _rand((B,), device, torch.float32,
                                          name + ".in", 2.5 / B))
        self.outw = _param(1.0 + _rand((B,), device, torch.float32,
                                       name + ".out", 2.5))
        self.mix = _param(torch.eye(B, device=device) + _rand(
            (B, B), device, torch.float32, name + ".mix", 2.5 / B))

    def step(self, streams, y, hc, norm_w, eps, dtype):
        """Write the previous sublayer's result y through its weights hc
        (None before the first sublayer), read this sublayer's input."""
        mix, outw = (None, None) if y is None else (hc.mix, hc.outw)
        return ops.stream_step(streams, y, mix, outw, self.inw, norm_w, eps,
                               dtype)


class StreamLayer(nn.Module):
    def __init__(self, cfg: DefosunConfig, i: int, device, dtype):
        super().__init__()
        spec = cfg.layers[i]
        D, eps = cfg.hidden_size, cfg.norm_eps
        self.eps, self.dtype = eps, dtype
        name = f"l{i}.mix"
        if spec.type == "attention":
            self.mixer = SinkRotaryAttention(D, spec.mixer, eps, name,
                                             device, dtype)
        elif spec.type == "latent_attention":
            self.mixer = LatentAttention(D, spec.mixer, eps, name, device,
                                         dtype)
        elif spec.type == "lightning":
            self.mixer = FixedDecayAttention(D, spec.mixer, eps, name,
                                             device, dtype)
        else:
            raise ValueError(f"layer {i}: unknown mixer {spec.type!r}")
        # norm weights are held as 1 + stored weight
        self.norm1_w = _norm_w(D, device, f"l{i}.norm1")
        self.hc1 = StreamMix(cfg.streams, f"l{i}.hc1", device)
        self.norm2_w = self.hc2 = self.mlp = None
        if spec.mlp is None:
            return
        self.norm2_w = _norm_w(D, device, f"l{i}.norm2")
        self.hc2 = StreamMix(cfg.streams, f"l{i}.hc2", device)
        if isinstance(spec.mlp, SiluFFSpec):
            self.mlp = GatedMLP(D, spec.mlp, f"l{i}.mlp", device, dtype,
                                ops.GATED_ACT_SILU)
        else:
            self.mlp = SharedExpertMoE(D, spec.mlp, f"l{i}.mlp", device,
                                       dtype)

    def cache_spec(self) -> tuple:
        s = self.mixer.cache_spec()
        return ("group", s) if isinstance(s, list) else s

    def forward(self, streams, y, hc, fb, cache):
        """(y, hc): the PREVIOUS sublayer's result and its stream weights,
        written into the streams by this sublayer's first kernel.  Returns
        (streams, this layer's last unwritten pair)."""
        streams, h = self.hc1.step(streams, y, hc, self.norm1_w, self.eps,
                                   self.dtype)
        y, hc = self.mixer(h, fb, cache), self.hc1
        if self.mlp is not None:
            streams, h = self.hc2.step(streams, y, hc, self.norm2_w,
                                       self.eps, self.dtype)
            y, hc = self.mlp(h, fb), self.hc2
        return streams, y, hc


class DefosunForCausalLM(nn.Module):
    needs_seq_meta = True          # ForwardBatch.seq_* / row_seq fields
    supports_decode_graph = False  # decode runs eagerly
    supported_dtypes = (torch.bfloat16, torch.float32)

    def __init__(self, cfg: DefosunConfig, device, dtype=torch.bfloat16):
        super().__init__()
        if tp_world_size() != 1:
            raise ValueError("Defosun runs unsharded (tensor parallel "
                             "degree 1)")
        self.cfg = cfg
        self.device = device
        self.dtype = dtype
        D = cfg.hidden_size
        self.embed = _param(_rand((cfg.vocab_size, D), device, dtype,
                                  "embed", 50.0))
        self.layers = nn.ModuleList(
            StreamLayer(cfg, i, device, dtype)
            for i in range(cfg.num_layers))
        self.final_norm_w = _norm_w(D, device, "final.norm")
        self.head = _w((cfg.vocab_size, D), device, dtype, "head", D)
        self.runs = cfg.layer_runs
        self.register_buffer("stream_sum", torch.ones(
            cfg.streams, dtype=torch.float32, device=device),
            persistent=False)
        self.tap = None    # debugging hook: called with (run, residual)

    def cache_specs(self) -> List[tuple]:
        """One entry per layer RUN (a repeated layer keeps a cache per
        pass): paged K/V, paged latent rows, or a slot's memory."""
        return [self.layers[i].cache_spec() for i in self.runs]

    def forward(self, fb: ForwardBatch, caches) -> torch.Tensor:
        cfg = self.cfg
        x = F.embedding(fb.token_ids, self.embed).float()
        streams = x.unsqueeze(1).expand(-1, cfg.streams, -1)
        y = hc = None
        for n, i in enumerate(self.runs):
            streams, y, hc = self.layers[i](streams, y, hc, fb, caches[n])
            if self.tap is not None:
                self.tap(n, (streams * hc.mix.sum(1)[None, :, None]).sum(1)
                         + hc.outw.sum() * y.float())
        return ops.stream_step(streams, y, hc.mix, hc.outw, self.stream_sum,
                               self.final_norm_w, cfg.norm_eps,
                               self.dtype)[1]

    def compute_logits(self, hidden_last: torch.Tensor) -> torch.Tensor:
        return F.linear(hidden_last, self.head).float()
