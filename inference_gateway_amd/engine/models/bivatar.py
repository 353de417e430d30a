"""Bivatar: a per-layer post-norm decoder for the MI355X engine.

The fp32 residual stream starts as the scaled token row.  The sublayers
read the stream itself; only their outputs are normed,

    x <- x + m norm1(mixer(x));   x <- x + m norm2(ff(x))

with RMS norms and one multiplier m.  Mixers, chosen per layer:

  WindowAttention   softmax attention without rotation: per-head q/k RMS
                    norm, a linear bias per head on the distance, keys from
                    a sliding window plus the sequence's first tokens, one
                    sigmoid output gate per head
  LatentAttention   low-rank queries and keys/values (engine/models/
                    fedatar.py) with half-split YaRN rotary positions and
                    the ordinary softmax; a layer may read ANOTHER layer's
                    cached latents with its own up-projections

The feed-forward is GatedMLP (gelu-gated).  Everything a layer keeps
between steps is paged and handed in by the engine (cache_specs), so
portions of prompts, decoded tokens and mixed batches are one code path.
GEMMs go through F.linear/bmm; everything between them is a gfx950 kernel
from ops, the residual update fused with its norm and the cast that the
next GEMM reads.
"""
from __future__ import annotations

from typing import List

import torch
import torch.nn as nn
import torch.nn.functional as F

from ... import ops
from ...parallel.comm import tp_world_size
from ..config import BivatarConfig, GatedFFSpec, WindowAttentionSpec
from .batch import ForwardBatch
from .bozolorn import _norm_w, _w
from .fedatar import LatentAttention, _param, _rand


class WindowAttention(nn.Module):
    """q, k RMS-normed per head (one weight vector shared by the heads);
    score(i, j) = q_i . k_j * scale - slope_h (i - j), slope_h =
    2^(-8 (h + 1) / H); j <= i and (i - j < window or j < keep_first);
    softmax; head h times sigmoid(W_g h)_h, then W_o."""

    def __init__(self, hidden: int, spec: WindowAttentionSpec, eps: float,
                 name: str, device, dtype):
        super().__init__()
        self.spec, self.eps = spec, eps
        H, G, N, P = spec.heads, spec.kv_heads, spec.dim, spec.vdim
        # fused projection rows: q | k | v | per-head gate logits
        self.gate0 = H * N + G * N + G * P
        self.qkvg = _w((self.gate0 + H, hidden), device, dtype,
                       name + ".qkvg", hidden)
        self.qnorm_w = _norm_w(N, device, name + ".q.norm")
        self.knorm_w = _norm_w(N, device, name + ".k.norm")
        self.o = _w((hidden, H * P), device, dtype, name + ".o", H * P)
        self.register_buffer("slopes", torch.tensor(
            [2.0 ** (-8.0 * (h + 1) / H) for h in range(H)],
            dtype=torch.float32, device=device)
            if spec.distance_bias else None, persistent=False)

    def cache_spec(self) -> tuple:
        s = self.spec
        return ("paged_k_v", s.kv_heads, s.dim, s.vdim)

    def forward(self, h: torch.Tensor, fb: ForwardBatch, cache):
        kc, vc = cache
        s = self.spec
        proj = F.linear(h, self.qkvg)
        q = ops.qk_norm_rope_append(
            proj, fb.positions, fb.slot_mapping, kc, vc, self.qnorm_w,
            self.knorm_w, None, 1.0, self.eps, s.heads, s.kv_heads, s.dim,
            s.vdim)
        o = ops.softcap_attention(
            q, kc, vc, fb.seq_block_table, fb.row_seq, fb.positions,
            s.scale, 0.0, 0.0, 1, s.window, fb.num_chunk_rows, fb.seq_lens,
            fb.seq_cu, fb.seq_start, slopes=self.slopes,
            gate=proj[:, self.gate0:], keep=s.keep_first)
        return F.linear(o, self.o)


class GatedMLP(nn.Module):
    """W_down (act(W_gate h) * (W_up h)); gate and up are one fused
    GEMM, `mode` is the activation of ops.gated_act."""

    def __init__(self, hidden: int, spec: GatedFFSpec, name: str, device,
                 dtype, mode: int = ops.GATED_ACT_GELU):
        super().__init__()
        self.mode = mode
        self.gate_up = _w((2 * spec.ff, hidden), device, dtype,
                          name + ".gate_up", hidden)
        self.down = _w((hidden, spec.ff), device, dtype, name + ".down",
                       spec.ff)

    def forward(self, h: torch.Tensor, fb: ForwardBatch) -> torch.Tensor:
        return F.linear(ops.gated_act(F.linear(h, self.gate_up), self.mode),
                        self.down)


class PostNormLayer(nn.Module):
    def __init__(self, cfg: BivatarConfig, i: int, device, dtype):
        super().__init__()
        spec = cfg.layers[i]
        D, eps = cfg.hidden_size, cfg.norm_eps
        self.eps, self.mult, self.dtype = eps, cfg.residual_mult, dtype
        name = f"l{i}.mix"
        self.kv_from = -1
        if spec.type == "attention":
            self.mixer = WindowAttention(D, spec.mixer, eps, name, device,
                                         dtype)
        elif spec.type == "latent_attention":
            self.mixer = LatentAttention(D, spec.mixer, eps, name, device,
                                         dtype)
            self.kv_from = spec.mixer.kv_from
        else:
            raise ValueError(f"layer {i}: unknown mixer {spec.type!r}")
        self.norm1_w = _norm_w(D, device, f"l{i}.norm1")
        if spec.mlp is None:
            self.norm2_w = self.mlp = None
        else:
            self.norm2_w = _norm_w(D, device, f"l{i}.norm2")
            self.mlp = GatedMLP(D, spec.mlp, f"l{i}.mlp", device, dtype)

    def forward(self, residual, delta, w_post, fb, cache):
        """residual: fp32 stream; (delta, w_post): the PREVIOUS
        sublayer's output and the weight of its norm, added inside this
        sublayer's fused residual kernel.  Returns this layer's last
        un-added pair."""
        x = ops.add_normed_rmsnorm(residual, delta, w_post, None, self.eps,
                                   self.dtype, self.mult)
        delta, w_post = self.mixer(x, fb, cache), self.norm1_w
        if self.mlp is not None:
            x = ops.add_normed_rmsnorm(residual, delta, w_post, None,
                                       self.eps, self.dtype, self.mult)
            delta, w_post = self.mlp(x, fb), self.norm2_w
        return delta, w_post


class BivatarForCausalLM(nn.Module):
    needs_seq_meta = True          # ForwardBatch.seq_* / row_seq fields
    supports_decode_graph = False  # decode runs eagerly
    supported_dtypes = (torch.bfloat16, torch.float32)

    def __init__(self, cfg: BivatarConfig, device, dtype=torch.bfloat16):
        super().__init__()
        if tp_world_size() != 1:
            raise ValueError("Bivatar runs unsharded (tensor parallel "
                             "degree 1)")
        self.cfg = cfg
        self.device = device
        self.dtype = dtype
        D = cfg.hidden_size
        self.embed = _param(_rand((cfg.vocab_size, D), device, dtype,
                                  "embed", 50.0 / cfg.embed_scale))
        self.layers = nn.ModuleList(
            PostNormLayer(cfg, i, device, dtype)
            for i in range(cfg.num_layers))
        self.final_norm_w = _norm_w(D, device, "final.norm")
        self.head = _w((cfg.vocab_size, D), device, dtype, "head", D)
        self.tap = None    # debugging hook: called with (layer, residual)

    def cache_specs(self) -> List[tuple]:
        """One entry per layer: paged K/V for windowed attention, paged
        latent rows for latent attention, nothing for a layer that reads
        another layer's."""
        return [l.mixer.cache_spec() for l in self.layers]

    def forward(self, fb: ForwardBatch, caches) -> torch.Tensor:
        cfg = self.cfg
        residual = F.embedding(fb.token_ids, self.embed).float()
        if cfg.embed_scale != 1.0:
            residual.mul_(cfg.embed_scale)
        delta = w_post = None
        for i, layer in enumerate(self.layers):
            cache = caches[layer.kv_from if layer.kv_from >= 0 else i]
            delta, w_post = layer(residual, delta, w_post, fb, cache)
            if self.tap is not None:
                d = delta.float()
                self.tap(i, residual + cfg.residual_mult * d * torch.rsqrt(
                    (d * d).mean(-1, keepdim=True) + cfg.norm_eps) * w_post)
        return ops.add_normed_rmsnorm(
            residual, delta, w_post, self.final_norm_w, cfg.norm_eps,
            self.dtype, cfg.residual_mult)

    def compute_logits(self, hidden_last: torch.Tensor) -> torch.Tensor:
        return F.linear(hidden_last, self.head).float()
