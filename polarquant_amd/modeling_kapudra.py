"""Kapudra: a decoder of parallel layers whose mixer is windowed attention beside a gated delta rule, or a matrix memory;
some layers run several times with the same weights.  Described layer by layer in its config.json."""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional, Tuple, Union

import torch.nn as nn

from .modeling_recurrent import (GatedDelta, GatedGelu, Loop, MatrixMemory, ParallelLayer, RecurrentForCausalLM, RecurrentModel, SideBySide,
                                 WindowAttention, distance_slopes)


@dataclass
class WindowMixerConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    window: int
    scale: float


@dataclass
class DeltaMixerConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    decay_rank: Optional[int] = None        # the ranks of the decay's and the gate's products: a checkpoint's shapes tell
    gate_rank: Optional[int] = None


@dataclass
class ParallelMixerConfig:
    left: WindowMixerConfig
    right: DeltaMixerConfig
    left_scale: float
    right_scale: float


@dataclass
class MemoryMixerConfig:
    heads: int
    dim: int
    vdim: int
    gate_cap: float


@dataclass
class KapudraLayerConfig:
    mixer: Union[ParallelMixerConfig, MemoryMixerConfig]
    ff: Optional[int] = None                # None: the layer has no feed-forward


def _take(d: Dict, where: str, **kinds) -> Dict:
    """The named entries of d, converted; anything else in it is refused."""
    unknown = sorted(set(d) - set(kinds))
    if unknown:
        raise ValueError("polarquant_amd: %s has options that are not implemented: %s" % (where, unknown))
    return {k: kind(d[k]) for k, kind in kinds.items()}


def _mixer(i: int, entry: Dict):
    m, where = entry["mixer"], "layer %d's mixer" % i
    if entry["type"] == "mlstm":
        return MemoryMixerConfig(**_take(m, where, heads=int, dim=int, vdim=int, gate_cap=float))
    if entry["type"] != "parallel":
        raise ValueError("polarquant_amd: layer %d has mixer type %r; this design has parallel and mlstm" % (i, entry["type"]))
    m = _take(m, where, left=dict, right=dict, left_scale=float, right_scale=float)
    left = _take(m["left"], where + " (left)", heads=int, kv_heads=int, dim=int, vdim=int, scale=float, mask=dict)
    window = _take(left.pop("mask"), where + " (left mask)", size=int)["size"]
    right = _take(m["right"], where + " (right)", heads=int, kv_heads=int, dim=int, vdim=int, conv=int)
    return ParallelMixerConfig(WindowMixerConfig(window=window, **left), DeltaMixerConfig(**right), m["left_scale"], m["right_scale"])


@dataclass
class KapudraConfig:
    vocab_size: int
    hidden_size: int
    layers: List[KapudraLayerConfig]
    norm_eps: float
    embedding_scale: float = 1.0
    logit_scale: float = 1.0
    logit_softcap: Optional[float] = None
    loop: Optional[Loop] = None
    eos_token_id: List[int] = field(default_factory=list)
    cache_capacity: int = 0             # (the state does not grow with the sequence)
    tie_word_embeddings: bool = False

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @staticmethod
    def from_dict(d: Dict, cache_capacity: int = 0) -> "KapudraConfig":
        """From the dict of a checkpoint's config.json."""
        layers: List[KapudraLayerConfig] = []
        for i, entry in enumerate(d["layers"]):
            mlp = entry.get("mlp")
            if mlp is not None and mlp.get("kind") != "dense":
                raise ValueError("polarquant_amd: layer %d has a feed-forward of kind %r; this design has dense" % (i, mlp.get("kind")))
            layers.append(KapudraLayerConfig(_mixer(i, entry), None if mlp is None else int(mlp["ff"])))
        loop = d.get("loop")
        if loop is not None:
            loop = Loop(**_take(loop, "the loop", start=int, stop=int, times=int))
            if not (0 <= loop.start < loop.stop <= len(layers) and loop.times >= 1):
                raise ValueError("polarquant_amd: no loop over layers %d .. %d of %d, %d times" % (loop.start, loop.stop - 1, len(layers), loop.times))
        eos = d.get("eos_token_id")
        eos = [] if eos is None else [int(e) for e in eos] if isinstance(eos, (list, tuple)) else [int(eos)]
        cap = d.get("logit_softcap")
        return KapudraConfig(vocab_size=d["vocab"], hidden_size=d["width"], layers=layers, norm_eps=float(d["norm"]["eps"]),
                             embedding_scale=float(d["embedding"]["scale"]), logit_scale=float(d["logit_scale"]),
                             logit_softcap=None if cap is None else float(cap), loop=loop, eos_token_id=eos, cache_capacity=cache_capacity)

    def to_dict(self) -> Dict:
        def entry(l):
            m = l.mixer
            mlp = None if l.ff is None else {"ff": l.ff, "kind": "dense"}
            if isinstance(m, MemoryMixerConfig):
                return {"type": "mlstm", "mixer": {k: getattr(m, k) for k in ("dim", "gate_cap", "heads", "vdim")}, "mlp": mlp}
            left = dict({k: getattr(m.left, k) for k in ("dim", "heads", "kv_heads", "scale", "vdim")}, mask={"size": m.left.window})
            right = {k: getattr(m.right, k) for k in ("conv", "dim", "heads", "kv_heads", "vdim")}
            return {"type": "parallel", "mixer": {"left": left, "left_scale": m.left_scale, "right": right, "right_scale": m.right_scale}, "mlp": mlp}
        d = {"architecture": "Kapudra", "embedding": {"scale": self.embedding_scale}, "layers": [entry(l) for l in self.layers],
             "logit_scale": self.logit_scale, "logit_softcap": self.logit_softcap,
             "loop": None if self.loop is None else {"start": self.loop.start, "stop": self.loop.stop, "times": self.loop.times},
             "norm": {"eps": self.norm_eps}, "vocab": self.vocab_size, "width": self.hidden_size}
        if self.eos_token_id:
            d["eos_token_id"] = self.eos_token_id
        return d

    def take_shapes(self, shapes: Dict[str, Tuple[int, ...]]) -> None:
        """Sizes that only a checkpoint's tensors tell: the ranks of the delta rules' low-rank products."""
        for i, l in enumerate(self.layers):
            if isinstance(l.mixer, ParallelMixerConfig):
                for attr, name in (("decay_rank", "a1"), ("gate_rank", "g1")):
                    full = "l%d.mix.right.%s" % (i, name)
                    if full not in shapes:
                        raise KeyError("polarquant_amd: the checkpoint has no tensor for %s" % full)
                    setattr(l.mixer.right, attr, int(shapes[full][0]))


class KapudraModel(RecurrentModel):
    def build_layers(self, config: KapudraConfig):
        W, eps = config.hidden_size, config.norm_eps
        for i, l in enumerate(config.layers):
            m = l.mixer
            if isinstance(m, MemoryMixerConfig):
                mix = MatrixMemory(W, m.heads, m.dim, m.vdim, m.gate_cap, eps)
            else:
                a, r = m.left, m.right
                if r.decay_rank is None or r.gate_rank is None:
                    raise ValueError("polarquant_amd: layer %d's low-rank products have no ranks yet (KapudraConfig.take_shapes)" % i)
                mix = SideBySide(WindowAttention(W, a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.scale, eps, distance_slopes(a.heads), m.left_scale),
                                 GatedDelta(W, r.heads, r.kv_heads, r.dim, r.vdim, r.conv, r.decay_rank, r.gate_rank, eps, m.right_scale))
            yield ParallelLayer(mix, None if l.ff is None else GatedGelu(W, l.ff), W, eps)


class KapudraForCausalLM(RecurrentForCausalLM):
    model_class = KapudraModel

    def checkpoint_tensors(self) -> Dict[str, nn.Parameter]:
        """Checkpoint tensor name -> parameter."""
        m = self.model
        out = {"embed": m.embed_tokens.weight, "final.norm": m.norm.weight, "head": self.lm_head.weight}
        if m.loop_step is not None:
            out["loop.step"] = m.loop_step
        for i, layer in enumerate(m.layers):
            out["l%d.norm1" % i] = layer.norm1.weight
            for part in ("mix", "mlp"):
                sub = getattr(layer, part)
                if sub is not None:
                    out.update(("l%d.%s.%s" % (i, part, name), p) for name, p in sub.checkpoint_tensors())
        return out
