"""Decoder layers of parallel branches, with windowed attention and recurrent mixers: the mechanisms, their state, and the
model that runs them.

Mechanisms, each a module with its constants as arguments: `WindowAttention` (grouped heads, q and k normed over the whole
projection, a sliding window, a bias per position of distance), `GatedDelta` (gated delta rule with a decay per head and key
channel, short convolutions), `MatrixMemory` (exponentially gated matrix memory), `GatedGelu` (feed-forward), `SideBySide`
(mixers whose weighted results are added), `ParallelLayer` (one norm, every sublayer reads it), `Loop` (layers run several times
with the same weights, each pass with a state of its own).

All branches of a layer read one normed input and their results are summed, so a layer is two matrix products: one of all
input projections, and one of all output projections, whose operand the branches write side by side.  The residual stream
is float32 whatever the model's dtype.

The state of a layer run does not grow with the sequence: the window's ring, convolution inputs, matrices.  Its cache tuple
is `(tensors of each branch ..., kv_seq_len)`.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Iterator, List, Optional, Sequence, Tuple

import torch
import torch.nn as nn

from . import layer_ops
from . import recurrent_ops as ops
from .modeling_common import PolarCache
from .modeling_layered import LayeredForCausalLM, LayeredModel
from .recurrent_ops import Step

ALIGN = 8                  # elements: a branch's columns begin at multiples of 16 bytes


def _up(n: int, to: int) -> int:
    return -(-n // to) * to


def _weight(*shape) -> nn.Parameter:
    return nn.Parameter(torch.empty(*shape).normal_(0.0, 0.02))


class Packed:
    """Parameters as slices of one matrix, stacked along `axis`, each in as many rows (columns) as it is given, the rest
    zero; made again when a parameter has moved."""

    def __init__(self, pieces: Sequence[Tuple[nn.Parameter, int]], axis: int, total_to: int):
        self.pieces, self.axis, self.total_to = list(pieces), axis, total_to
        self._w: Optional[torch.Tensor] = None
        self._at: List[int] = []

    def weight(self) -> torch.Tensor:
        if self._w is None or any(p.data_ptr() != at for (p, _), at in zip(self.pieces, self._at)):
            total, first = _up(sum(n for _, n in self.pieces), self.total_to), self.pieces[0][0]
            shape = list(first.shape)
            shape[self.axis] = total
            w = torch.zeros(shape, dtype=first.dtype, device=first.device)
            o = 0
            for p, n in self.pieces:
                part = w.narrow(self.axis, o, p.shape[self.axis])
                part.copy_(p.data)
                p.data = part
                o += n
            self._w, self._at = w, [p.data_ptr() for p, _ in self.pieces]
        return self._w


# ----------------------------------------------------------------------------- state
class LayerArena:
    """The states of one layer run's branches for B sequences; `states` have tensors(), carried() and reset()."""

    def __init__(self, states: Sequence):
        self.states = [s for s in states if s is not None]
        self.by_branch = list(states)
        self.kv_len = 0
        self.start: Optional[torch.Tensor] = None       # int32 [B]: left padding of each sequence

    def reserve(self, tokens: int) -> None:
        pass                                            # (nothing grows)

    def reset(self) -> None:
        """The sequences end; the memory serves the next ones."""
        self.kv_len, self.start = 0, None
        for s in self.states:
            s.reset()

    def load(self, parts, n: int) -> None:
        mine = [t for s in self.states for t in s.tensors()]
        for t, p in zip(mine, parts):
            t.copy_(p)
        self.kv_len = n

    def step_state(self) -> List[torch.Tensor]:
        return [t for s in self.states for t in s.carried()]

    def as_tuple(self) -> PolarCache:
        return PolarCache(tuple(t for s in self.states for t in s.tensors()) + (self.kv_len,), self)


class WindowState(ops.WindowRing):
    def tensors(self):
        return [self.k, self.v]

    def carried(self):
        return []                                       # (a step writes the same row again)

    def reset(self):
        pass                                            # (rows that a sequence has not written are outside its windows)


class DeltaState:
    def __init__(self, B: int, heads: int, dim: int, vdim: int, taps: int, channels: int, device):
        self.conv = layer_ops.ConvState(B, taps, channels, device)
        self.S = torch.zeros(B, heads, vdim, dim, dtype=torch.float32, device=device)

    def tensors(self):
        return [self.conv.rows, self.S]

    carried = tensors

    def reset(self):
        self.conv.reset()
        self.S.zero_()


class MemoryState:
    def __init__(self, B: int, heads: int, dim: int, vdim: int, device):
        self.S, self.m = ops.memory_state(B, heads, dim, vdim, device)

    def tensors(self):
        return [self.S, self.m]

    carried = tensors

    def reset(self):
        self.S.zero_()
        self.m.zero_()


# ----------------------------------------------------------------------------- branches
class Branch(nn.Module):
    """A sublayer that reads its columns of the layer's input product and writes its columns of the output product's operand."""

    names = {}                                          # attribute -> checkpoint name, where they differ

    def ins(self) -> List[Tuple[nn.Parameter, int]]:
        """Input projections [n, width], with the columns given to each."""
        raise NotImplementedError

    def out_weight(self) -> nn.Parameter:
        raise NotImplementedError

    def new_state(self, B: int, dtype, device):
        return None

    def forward(self, p: List[torch.Tensor], out: torch.Tensor, state, step: Step) -> None:
        """p: rows of each input projection, their padding included; out: rows to fill."""
        raise NotImplementedError

    def branches(self) -> List["Branch"]:
        return [self]

    def checkpoint_tensors(self) -> Iterator[Tuple[str, nn.Parameter]]:
        for name, p in self.named_parameters():
            yield self.names.get(name, name), p


def distance_slopes(heads: int) -> torch.Tensor:
    """2^(-8 (h + 1) / heads) for head h."""
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)], dtype=torch.float32)


class WindowAttention(Branch):
    """softmax over the last `window` positions of scale q.k - slope_h * distance; q and k normed over the whole projection."""

    names = {"q_norm": "q.norm", "k_norm": "k.norm"}

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, window: int, scale: float, eps: float,
                 slopes: Optional[torch.Tensor] = None, out_scale: float = 1.0):
        super().__init__()
        if heads % kv_heads:
            raise ValueError("polarquant_amd: %d query heads do not share %d key heads evenly" % (heads, kv_heads))
        self.heads, self.kv_heads, self.dim, self.vdim, self.window = heads, kv_heads, dim, vdim, window
        self.scale, self.eps, self.slopes, self.out_scale = scale, eps, slopes, out_scale
        self.q, self.k, self.v = _weight(heads * dim, width), _weight(kv_heads * dim, width), _weight(kv_heads * vdim, width)
        self.q_norm, self.k_norm = nn.Parameter(torch.ones(heads * dim)), nn.Parameter(torch.ones(kv_heads * dim))
        self.o = _weight(width, heads * vdim)

    def ins(self):
        return [(w, _up(w.shape[0], ALIGN)) for w in (self.q, self.k, self.v)]

    def out_weight(self):
        return self.o

    def new_state(self, B, dtype, device):
        if self.slopes is not None:
            self.slopes = self.slopes.to(device)        # (before a graph is captured)
        return WindowState(B, self.kv_heads, self.dim, self.vdim, self.window, dtype, device)

    def forward(self, p, out, state, step):
        q, k, v = [x[:, :w.shape[0]] for x, w in zip(p, (self.q, self.k, self.v))]
        q, k = ops.qk_norm(q, k, v, self.q_norm, self.k_norm, self.heads, self.eps, state, step)
        ops.window_attention(q, state, self.slopes, self.scale, step, out, self.out_scale, k, None if k is None else v)


class GatedDelta(Branch):
    """Per head S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q with unit q, k after short convolutions and silu; decays
    g per key channel and output gates through low-rank products."""

    names = {"q_conv": "q.conv", "k_conv": "k.conv", "v_conv": "v.conv"}

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, taps: int, decay_rank: int, gate_rank: int, eps: float,
                 out_scale: float = 1.0):
        super().__init__()
        if heads % kv_heads:
            raise ValueError("polarquant_amd: %d value heads do not share %d key heads evenly" % (heads, kv_heads))
        if max(dim, vdim) > ops.MAX_DIM or not 1 <= taps <= ops.MAX_TAPS:
            raise ValueError("polarquant_amd: a recurrent head of %d x %d or a convolution of %d taps is larger than the kernels take" % (dim, vdim, taps))
        self.heads, self.kv_heads, self.dim, self.vdim, self.taps, self.eps, self.out_scale = heads, kv_heads, dim, vdim, taps, eps, out_scale
        kd, vd = kv_heads * dim, heads * vdim
        self.q, self.k, self.v = _weight(kd, width), _weight(kd, width), _weight(vd, width)
        self.q_conv, self.k_conv, self.v_conv = _weight(kd, taps), _weight(kd, taps), _weight(vd, taps)
        self.b, self.A_log, self.norm = _weight(heads, width), nn.Parameter(torch.zeros(heads)), nn.Parameter(torch.ones(vdim))
        self.a1, self.a2, self.dt_bias = _weight(decay_rank, width), _weight(heads * dim, decay_rank), nn.Parameter(torch.zeros(heads * dim))
        self.g1, self.g2 = _weight(gate_rank, width), _weight(vd, gate_rank)
        self.o = _weight(width, vd)
        # the ranks in multiples of 32, so that the second products run the small-batch kernels too
        self._a2, self._g2 = Packed([(self.a2, _up(decay_rank, 32))], 1, 32), Packed([(self.g2, _up(gate_rank, 32))], 1, 32)

    def ins(self):
        return [(w, _up(w.shape[0], ALIGN)) for w in (self.q, self.k, self.v, self.b)] + [(w, _up(w.shape[0], 32)) for w in (self.a1, self.g1)]

    def out_weight(self):
        return self.o

    def new_state(self, B, dtype, device):
        return DeltaState(B, self.heads, self.dim, self.vdim, self.taps, 2 * self.kv_heads * self.dim + self.heads * self.vdim, device)

    def forward(self, p, out, state, step):
        q, k, v, b = [x[:, :w.shape[0]] for x, w in zip(p, (self.q, self.k, self.v, self.b))]
        a, gate = layer_ops.linear(p[4], self._a2.weight()), layer_ops.linear(p[5], self._g2.weight())
        x = ops.delta_prep(q, k, v, b, a, self.q_conv, self.k_conv, self.v_conv, self.A_log, self.dt_bias, state.conv, self.dim, self.vdim, step)
        ops.head_norm_gate(ops.delta_scan(x, state.S, step), self.norm, gate, self.heads, self.eps, out, self.out_scale)


class MatrixMemory(Branch):
    """Per head S <- f S + i k v^T, n <- f n + i k with exponential gates relative to a running maximum, read out as
    S^T q / max(|n.q|, e^-m); gates capped before they are exponentiated."""

    names = {"i_b": "i.b", "f_b": "f.b"}

    def __init__(self, width: int, heads: int, dim: int, vdim: int, gate_cap: float, eps: float, out_scale: float = 1.0):
        super().__init__()
        if dim > ops.MAX_DIM:
            raise ValueError("polarquant_amd: a recurrent head of %d channels is larger than the kernels take" % dim)
        self.heads, self.dim, self.vdim, self.gate_cap, self.eps, self.out_scale = heads, dim, vdim, gate_cap, eps, out_scale
        qd, vd = heads * dim, heads * vdim
        self.q, self.k, self.v, self.g, self.o = _weight(qd, width), _weight(qd, width), _weight(vd, width), _weight(vd, width), _weight(width, vd)
        self.norm = nn.Parameter(torch.ones(vd))
        self.i, self.i_b, self.f, self.f_b = _weight(heads, width), nn.Parameter(torch.zeros(heads)), _weight(heads, width), nn.Parameter(torch.zeros(heads))

    def ins(self):
        return [(w, _up(w.shape[0], ALIGN)) for w in (self.q, self.k, self.v, self.g, self.i, self.f)]

    def out_weight(self):
        return self.o

    def new_state(self, B, dtype, device):
        return MemoryState(B, self.heads, self.dim, self.vdim, device)

    def forward(self, p, out, state, step):
        q, k, v, g, i, f = [x[:, :w.shape[0]] for x, w in zip(p, (self.q, self.k, self.v, self.g, self.i, self.f))]
        log_i, log_f = ops.memory_gates(i, f, self.i_b, self.f_b, self.gate_cap)
        o, den = ops.memory_scan(q, k, v, log_i, log_f, state.S, state.m, self.dim ** -0.5, step)
        ops.head_norm_gate(o, self.norm, g, self.heads, self.eps, out, self.out_scale, den)


class GatedGelu(Branch):
    """W_down (gelu(W_gate h) * (W_up h)), the tanh form of gelu."""

    def __init__(self, width: int, ff: int):
        super().__init__()
        self.gate, self.up, self.down = _weight(ff, width), _weight(ff, width), _weight(width, ff)

    def ins(self):
        return [(w, _up(w.shape[0], ALIGN)) for w in (self.gate, self.up)]

    def out_weight(self):
        return self.down

    def forward(self, p, out, state, step):
        n = self.gate.shape[0]
        layer_ops.gelu_mul(p[0][:, :n], p[1][:, :n], out)


class SideBySide(nn.Module):
    """Two mixers that read the same input; their results are added (each scales its own)."""

    def __init__(self, left: Branch, right: Branch):
        super().__init__()
        self.left, self.right = left, right

    def branches(self):
        return [self.left, self.right]

    def checkpoint_tensors(self):
        for side in ("left", "right"):
            for name, p in getattr(self, side).checkpoint_tensors():
                yield side + "." + name, p


class RMSNorm(nn.Module):
    """Weight and constant of weight * x / rms(x); the arithmetic is part of the launches that use it."""

    def __init__(self, width: int, eps: float):
        super().__init__()
        self.weight, self.eps = nn.Parameter(torch.ones(width)), eps


class ParallelLayer(nn.Module):
    """x <- x + (mixer(norm(x)) + mlp(norm(x)))."""

    def __init__(self, mixer: nn.Module, mlp: Optional[Branch], width: int, eps: float):
        super().__init__()
        self.norm1, self.mix, self.mlp = RMSNorm(width, eps), mixer, mlp
        self._branches = mixer.branches() + ([] if mlp is None else mlp.branches())
        self._in = Packed([piece for br in self._branches for piece in br.ins()], 0, 16)
        self._out = Packed([(w, _up(w.shape[1], ALIGN)) for w in (br.out_weight() for br in self._branches)], 1, 32)

    def new_arena(self, B: int, dtype, device) -> LayerArena:
        return LayerArena([br.new_state(B, dtype, device) for br in self._branches])

    def forward(self, h: torch.Tensor, arena: LayerArena, step: Step) -> torch.Tensor:
        """h [B, L, width], normed -> what is added to the stream."""
        w_in, w_out = self._in.weight(), self._out.weight()
        M = step.B * step.L
        p = layer_ops.linear(h.view(M, -1), w_in)
        K = w_out.shape[1]
        filled = sum(w.shape[1] for w in (br.out_weight() for br in self._branches)) == K
        z = (torch.empty if filled else torch.zeros)(M, K, dtype=h.dtype, device=h.device)
        at = col = 0
        for br, state in zip(self._branches, arena.by_branch):
            rows = []
            for _, n in br.ins():
                rows.append(p[:, at:at + n])
                at += n
            k = br.out_weight().shape[1]
            br(rows, z[:, col:col + k], state, step)
            col += _up(k, ALIGN)
        return layer_ops.linear(z, w_out).view(step.B, step.L, -1)


@dataclass
class Loop:
    """Layers start .. stop - 1 run `times` times in a row."""
    start: int
    stop: int
    times: int


def layer_runs(layers: int, loop: Optional[Loop]) -> List[Tuple[int, Optional[int]]]:
    """(layer, number of the pass that begins with it or None) in the order of running."""
    if loop is None or loop.stop <= loop.start:
        return [(i, None) for i in range(layers)]
    passes = [(i, t if i == loop.start else None) for t in range(loop.times) for i in range(loop.start, loop.stop)]
    return [(i, None) for i in range(loop.start)] + passes + [(i, None) for i in range(loop.stop, layers)]


# ----------------------------------------------------------------------------- model
class RecurrentModel(LayeredModel):
    """Scaled embedding, parallel layers (some of them looped), final norm.  Before a pass of the loop a vector of its own is
    added to the stream, and before every pass but the first the embedding once more."""

    def __init__(self, config):
        super().__init__(config)
        self.norm = RMSNorm(config.hidden_size, config.norm_eps)
        self.runs = layer_runs(len(self.layers), config.loop)
        self.loop_step = nn.Parameter(torch.zeros(config.loop.times, config.hidden_size)) if config.loop is not None else None

    def new_arenas(self, B: int, capacity: int) -> List[LayerArena]:
        w = self.embed_tokens.weight
        return [self.layers[i].new_arena(B, w.dtype, w.device) for i, _ in self.runs]

    def run(self, input_ids, arenas, pos, pos_dev=None, plan=None):
        B, L = input_ids.shape
        step = Step(B, L, pos, pos_dev, arenas[0].start if arenas else None)
        norm = lambda x, n, y: layer_ops.norm_conv(x, n.weight, 1, n.eps, y, start=step.start, pos=pos, pos_dev=pos_dev)
        e = layer_ops.embed_rows(self.embed_tokens.weight, input_ids, self.config.embedding_scale)
        again = any(t for _, t in self.runs)            # the embedding is needed later, and short calls norm in place
        x, y = (e.clone() if again and self.runs[0][1] is None else e), None
        for (i, t), arena in zip(self.runs, arenas):
            if t is not None:
                x, y = layer_ops.stream_add(x, y, e if t > 0 else None, self.loop_step[t]), None
            x, h = norm(x, self.layers[i].norm1, y)
            y = self.layers[i](h, arena, step)
            if self.capture is not None:
                self.capture.append(x + y.float())
        return norm(x, self.norm, y)[1]


class RecurrentForCausalLM(LayeredForCausalLM):
    model_class = RecurrentModel

    @torch.no_grad()
    def logits(self, h):
        return layer_ops.softcap(super().logits(h), self.config.logit_scale, self.config.logit_softcap)

    def kv_cache_bytes_per_token(self) -> int:
        """Nothing grows with the sequence (state_bytes counts what a sequence holds)."""
        return 0

    def state_bytes(self) -> int:
        """Bytes that one sequence holds, whatever its length."""
        return sum(t.numel() * t.element_size() for a in self.model.new_arenas(1, 1) for s in a.states for t in s.tensors())
