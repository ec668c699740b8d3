"""Decoder layers with latent attention: the mechanisms, their per-layer cache, and the model that runs them.

Mechanisms, each a module with its constants as arguments: `LatentAttention` (queries and a shared key/value latent
through low-rank projections, no positions, a per-head sink, an output gate, optionally the latent of an earlier layer),
`GroupRMSNorm`, `InputConv` (causal depthwise convolution added to a sublayer's input), `ReluSquaredMLP`, `SandwichLayer`
(norm before and after each sublayer).  The residual stream is float32 whatever the model's dtype.

The cache tuple of a layer is `(latents | None, mixer-convolution state, feed-forward-convolution state | None, kv_seq_len)`,
a `PolarCache` whose arena owns the tensors.
"""
from __future__ import annotations

from typing import List, Optional

import torch
import torch.nn as nn

from . import latent_ops as ops
from .modeling_common import PolarCache
from .modeling_layered import LayeredForCausalLM, LayeredModel

KEY_TILE = 64              # capacities are whole tiles of the prompt kernel's keys
ABSORBED_TOKENS = 16       # up to this many new tokens per sequence, queries go to the latent space instead of keys and values to the heads'


# ----------------------------------------------------------------------------- cache
class LatentArena:
    """Per-layer state of B sequences: the latents [B, capacity, kv_rank] (none in a layer that reads an earlier layer's,
    `source`), the two input convolutions' states, and the counts.  Rows from kv_len on are zero or left from an earlier
    use: finite, never attended to."""

    def __init__(self, B: int, kv_rank: int, taps: int, width: int, dtype, device, capacity: int, source: Optional["LatentArena"] = None,
                 has_mlp: bool = True):
        self.B, self.kv_rank, self.dtype, self.device, self.source = B, kv_rank, dtype, device, source
        self.conv = [ops.ConvState(B, taps, width, device) for _ in range(2 if has_mlp else 1)]
        self.kv_len = 0
        self.start: Optional[torch.Tensor] = None       # int32 [B]: left padding of each sequence
        self._c = None if source is not None else self._rows(capacity)

    def _rows(self, capacity: int) -> torch.Tensor:
        cap = -(-max(capacity, KEY_TILE) // KEY_TILE) * KEY_TILE
        return torch.zeros(self.B, cap, self.kv_rank, dtype=self.dtype, device=self.device)

    @property
    def c(self) -> torch.Tensor:
        return self._c if self.source is None else self.source.c

    def reserve(self, tokens: int) -> None:
        if self.source is None and tokens > self._c.shape[1]:
            new = self._rows(max(2 * self._c.shape[1], tokens))
            new[:, :self.kv_len] = self._c[:, :self.kv_len]
            self._c = new

    def reset(self) -> None:
        """The sequences end; the memory serves the next ones."""
        self.kv_len, self.start = 0, None
        for s in self.conv:
            s.reset()

    def load(self, parts, n: int) -> None:
        lat, *rows = parts
        self.kv_len = n
        if lat is not None:
            self._c[:, :n] = lat
        for state, r in zip(self.conv, rows):
            state.rows.copy_(r)

    def step_state(self) -> List[torch.Tensor]:
        return [s.rows for s in self.conv]

    def as_tuple(self) -> PolarCache:
        lat = self._c[:, :self.kv_len] if self.source is None else None
        return PolarCache((lat, self.conv[0].rows, self.conv[1].rows if len(self.conv) > 1 else None, self.kv_len), self)


# ----------------------------------------------------------------------------- mechanisms
class GroupRMSNorm(nn.Module):
    """weight * x, each of `groups` equal consecutive parts of x over its own root mean square; parameters only, the
    arithmetic is part of the launches that use it."""

    def __init__(self, width: int, groups: int, eps: float):
        super().__init__()
        if width % groups:
            raise ValueError("polarquant_amd: %d channels do not split into %d norm groups" % (width, groups))
        self.groups, self.eps = groups, eps
        self.weight = nn.Parameter(torch.ones(width))


class InputConv(nn.Module):
    """Taps of h + conv(h), weight [width, taps], the last tap on the current token."""

    def __init__(self, width: int, taps: int):
        super().__init__()
        self.weight = nn.Parameter(torch.zeros(width, taps))


class LatentAttention(nn.Module):
    """c_q = rmsnorm(W_dq h), q = W_uq c_q; c = rmsnorm(W_dkv h) (or the latent of layer `kv_from`), k = W_uk c, v = W_uv c
    per head; softmax(scale q k^T) with exp(sink) in the denominator; times sigmoid(W_g h); W_o."""

    def __init__(self, width: int, heads: int, dim: int, vdim: int, q_rank: int, kv_rank: int, scale: float, eps: float,
                 kv_from: Optional[int] = None):
        super().__init__()
        self.heads, self.dim, self.vdim, self.q_rank, self.kv_rank = heads, dim, vdim, q_rank, kv_rank
        self.scale, self.eps, self.kv_from = scale, eps, kv_from
        p = lambda *shape: nn.Parameter(torch.empty(*shape).normal_(0.0, 0.02))
        self.dq, self.dq_norm, self.uq = p(q_rank, width), nn.Parameter(torch.ones(q_rank)), p(heads * dim, q_rank)
        if kv_from is None:
            self.dkv, self.dkv_norm = p(kv_rank, width), nn.Parameter(torch.ones(kv_rank))
        self.uk, self.uv = p(heads * dim, kv_rank), p(heads * vdim, kv_rank)
        self.sink = nn.Parameter(torch.zeros(heads))
        self.g, self.o = p(heads * vdim, width), p(width, heads * vdim)
        self._fused = self._derived = None

    def _prepare(self):
        """The input projections as one matrix (the parameters become slices of it), W_uk with the head's latent as the
        output dimension, the sinks in float32; made again when a parameter has changed."""
        ins = [self.dq] + ([self.dkv] if self.kv_from is None else []) + [self.g]
        if self._fused is None or any(p.data_ptr() != at for p, at in zip(ins, self._fused[1])):
            w = torch.cat([p.data for p in ins], dim=0)
            o = 0
            for p in ins:
                p.data = w[o:o + p.shape[0]]
                o += p.shape[0]
            self._fused = (w, [p.data_ptr() for p in ins])
        key = (self.uk.data_ptr(), self.uk._version, self.sink.data_ptr(), self.sink._version)
        if self._derived is None or self._derived[0] != key:
            ukt = self.uk.data.view(self.heads, self.dim, self.kv_rank).transpose(1, 2).contiguous()
            self._derived = (key, ukt, self.sink.data.float().contiguous())
        return self._fused[0], self._derived[1], self._derived[2]

    def forward(self, h: torch.Tensor, arena: LatentArena, pos: int, pos_dev: Optional[torch.Tensor] = None,
                n_splits: Optional[int] = None) -> torch.Tensor:
        """h [B, L, width]; the tokens' positions are pos .. pos + L - 1 (*pos_dev .. when given, for replayed steps)."""
        B, L, _ = h.shape
        H, D, Dv, R = self.heads, self.dim, self.vdim, self.kv_rank
        w_in, ukt, sink = self._prepare()
        p = ops.linear(h, w_in)
        own = self.kv_from is None
        gate = p.view(B * L, -1)[:, self.q_rank + (R if own else 0):]
        c_q = ops.latent_norm(p, self.dq_norm, self.dkv_norm if own else None, arena.c if own else None, self.eps, pos, pos_dev)
        q = ops.linear(c_q, self.uq)
        c = arena.c
        if L <= ABSORBED_TOKENS or not ops.prefill_takes(D, Dv, q.dtype):
            q_lat = ops.head_linear(q.view(B * L, H, D), ukt)
            o_lat = ops.latent_decode_attention(q_lat.view(B, L, H, R), c, sink, self.scale, pos, pos_dev, arena.start, n_splits)
            o = ops.head_linear(o_lat.view(B * L, H, R), self.uv.view(H, Dv, R), gate=gate).view(B, L, H * Dv)
        else:
            Lk = pos + L
            ld = -(-Lk // KEY_TILE) * KEY_TILE
            k = torch.empty(B, Lk, H, D, dtype=q.dtype, device=q.device)
            vt = torch.empty(B, H, Dv, ld, dtype=q.dtype, device=q.device)
            for b in range(B):                  # (the values come out of the product with a row per channel)
                torch.mm(c[b, :Lk], self.uk.t(), out=k[b].view(Lk, H * D))
                torch.mm(self.uv, c[b, :ld].t(), out=vt[b].view(H * Dv, ld))
            o = ops.latent_prefill_attention(q.view(B, L, H, D), k, vt, sink, self.scale, gate, arena.start)
        return ops.linear(o, self.o)


class ReluSquaredMLP(nn.Module):
    def __init__(self, width: int, ff: int):
        super().__init__()
        self.up = nn.Parameter(torch.empty(ff, width).normal_(0.0, 0.02))
        self.down = nn.Parameter(torch.empty(width, ff).normal_(0.0, 0.02))

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        return ops.linear(ops.linear(h, self.up, relu_squared=True), self.down)


class SandwichLayer(nn.Module):
    """x <- x + post_norm(sublayer(conv(pre_norm(x)))) for the mixer and, if there is one, the feed-forward."""

    def __init__(self, mixer: nn.Module, mlp: Optional[nn.Module], width: int, groups: int, eps: float, taps: int):
        super().__init__()
        norm = lambda: GroupRMSNorm(width, groups, eps)
        self.mix, self.norm1, self.norm1b, self.canon1 = mixer, norm(), norm(), InputConv(width, taps)
        self.mlp = mlp
        if mlp is not None:
            self.norm2, self.norm2b, self.canon2 = norm(), norm(), InputConv(width, taps)

    def sublayers(self):
        yield self.norm1, self.canon1, self.mix, self.norm1b
        if self.mlp is not None:
            yield self.norm2, self.canon2, self.mlp, self.norm2b


# ----------------------------------------------------------------------------- model
class LatentModel(LayeredModel):
    """Layers with latent attention between an embedding and a final norm."""

    def __init__(self, config):
        super().__init__(config)
        self.norm = GroupRMSNorm(config.hidden_size, config.norm_groups, config.norm_eps)

    def new_arenas(self, B: int, capacity: int) -> List[LatentArena]:
        cfg, w = self.config, self.embed_tokens.weight
        arenas: List[LatentArena] = []
        for layer in self.layers:
            a = layer.mix
            arenas.append(LatentArena(B, a.kv_rank, cfg.canon_taps, cfg.hidden_size, w.dtype, w.device, capacity,
                                      None if a.kv_from is None else arenas[a.kv_from], layer.mlp is not None))
        return arenas

    def step_plan(self, B: int, max_len: int, device):
        return [ops.decode_splits(B, 1, layer.mix.heads, max_len, device) for layer in self.layers]

    def run(self, input_ids: torch.Tensor, arenas: List[LatentArena], pos: int, pos_dev: Optional[torch.Tensor] = None,
            plan: Optional[List[int]] = None) -> torch.Tensor:
        """plan: each layer's number of slices."""
        x = self.embed_tokens(input_ids).float()
        y = w_post = None
        start = arenas[0].start
        for i, (layer, arena) in enumerate(zip(self.layers, arenas)):
            for state, (pre, conv, sublayer, post) in zip(arena.conv, layer.sublayers()):
                first_of_layer = sublayer is layer.mix
                x, h = ops.norm_conv(x, pre.weight, pre.groups, pre.eps, y, w_post, conv.weight, state, start, pos, pos_dev)
                if first_of_layer and i and self.capture is not None:
                    self.capture.append(x.clone())
                if first_of_layer:
                    y = sublayer(h, arena, pos, pos_dev, None if plan is None else plan[i])
                else:
                    y = sublayer(h)
                w_post = post.weight
        x, h = ops.norm_conv(x, self.norm.weight, self.norm.groups, self.norm.eps, y, w_post, start=start, pos=pos, pos_dev=pos_dev)
        if self.capture is not None:
            self.capture.append(x.clone())
        return h


class LatentForCausalLM(LayeredForCausalLM):
    model_class = LatentModel

    def kv_cache_bytes_per_token(self) -> int:
        """Latents only: the convolutions' states do not grow with the sequence."""
        e = self.lm_head.weight.element_size()
        return sum(layer.mix.kv_rank * e for layer in self.model.layers if layer.mix.kv_from is None)
