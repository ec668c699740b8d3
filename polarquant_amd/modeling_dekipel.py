"""Dekipel: a decoder of latent-attention layers with norms on both sides of every sublayer, grouped RMS norms, input
convolutions, a squared-relu feed-forward and float32 residual stream, described layer by layer in its config.json."""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional

import torch.nn as nn

from .modeling_latent import LatentAttention, LatentForCausalLM, LatentModel, ReluSquaredMLP, SandwichLayer


@dataclass
class LatentMixerConfig:
    heads: int
    dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    kv_from: Optional[int] = None


@dataclass
class DekipelLayerConfig:
    mixer: LatentMixerConfig
    ff: Optional[int] = None            # None: the layer has no feed-forward


@dataclass
class DekipelConfig:
    vocab_size: int
    hidden_size: int
    layers: List[DekipelLayerConfig]
    norm_eps: float
    norm_groups: int
    canon_taps: int
    eos_token_id: List[int] = field(default_factory=list)
    cache_capacity: int = 0             # tokens to pre-allocate per layer (0: prompt + 1024, grown by doubling)
    tie_word_embeddings: bool = False

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @staticmethod
    def from_dict(d: Dict, cache_capacity: int = 0) -> "DekipelConfig":
        """From the dict of a checkpoint's config.json."""
        layers: List[DekipelLayerConfig] = []
        for i, entry in enumerate(d["layers"]):
            if entry["type"] != "latent_attention":
                raise ValueError("polarquant_amd: layer %d has mixer type %r; this design has latent_attention" % (i, entry["type"]))
            m = dict(entry["mixer"])
            mixer = LatentMixerConfig(heads=m.pop("heads"), dim=m.pop("dim"), vdim=m.pop("vdim"), q_rank=m.pop("q_rank"),
                                      kv_rank=m.pop("kv_rank"), scale=float(m.pop("scale")), kv_from=m.pop("kv_from", None))
            if m:
                raise ValueError("polarquant_amd: layer %d's mixer has options that are not implemented: %s" % (i, sorted(m)))
            j = mixer.kv_from
            if j is not None and not (0 <= j < i and layers[j].mixer.kv_from is None and layers[j].mixer.kv_rank == mixer.kv_rank):
                raise ValueError("polarquant_amd: layer %d takes its latents from layer %r, which has no latents of that rank of its own" % (i, j))
            mlp = entry.get("mlp")
            if mlp is not None and mlp.get("kind") != "dense":
                raise ValueError("polarquant_amd: layer %d has a feed-forward of kind %r; this design has dense" % (i, mlp.get("kind")))
            layers.append(DekipelLayerConfig(mixer, None if mlp is None else int(mlp["ff"])))
        eos = d.get("eos_token_id")
        eos = [] if eos is None else [int(e) for e in eos] if isinstance(eos, (list, tuple)) else [int(eos)]
        return DekipelConfig(vocab_size=d["vocab"], hidden_size=d["width"], layers=layers, norm_eps=float(d["norm"]["eps"]),
                             norm_groups=int(d["norm"]["groups"]), canon_taps=int(d["canon"]["taps"]), eos_token_id=eos,
                             cache_capacity=cache_capacity)

    def to_dict(self) -> Dict:
        def mixer(m):
            out = {k: getattr(m, k) for k in ("dim", "heads", "kv_rank", "q_rank", "scale", "vdim")}
            return out if m.kv_from is None else dict(out, kv_from=m.kv_from)
        d = {"architecture": "Dekipel", "canon": {"taps": self.canon_taps},
             "layers": [{"type": "latent_attention", "mixer": mixer(l.mixer), "mlp": None if l.ff is None else {"ff": l.ff, "kind": "dense"}}
                        for l in self.layers],
             "norm": {"eps": self.norm_eps, "groups": self.norm_groups}, "vocab": self.vocab_size, "width": self.hidden_size}
        if self.eos_token_id:
            d["eos_token_id"] = self.eos_token_id
        return d


class DekipelModel(LatentModel):
    def build_layers(self, config: DekipelConfig):
        W = config.hidden_size
        for l in config.layers:
            m = l.mixer
            mix = LatentAttention(W, m.heads, m.dim, m.vdim, m.q_rank, m.kv_rank, m.scale, config.norm_eps, m.kv_from)
            yield SandwichLayer(mix, None if l.ff is None else ReluSquaredMLP(W, l.ff), W, config.norm_groups, config.norm_eps,
                                config.canon_taps)


class DekipelForCausalLM(LatentForCausalLM):
    model_class = DekipelModel

    def checkpoint_tensors(self) -> Dict[str, nn.Parameter]:
        """Checkpoint tensor name -> parameter."""
        m = self.model
        out = {"embed": m.embed_tokens.weight, "final.norm": m.norm.weight, "head": self.lm_head.weight}
        for i, layer in enumerate(m.layers):
            l = "l%d." % i
            for name in ("norm1", "norm1b", "canon1", "norm2", "norm2b", "canon2"):
                if hasattr(layer, name):
                    out[l + name] = getattr(layer, name).weight
            for name, p in layer.mix.named_parameters():
                out[l + "mix." + name.replace("_norm", ".norm")] = p
            if layer.mlp is not None:
                out[l + "mlp.up"], out[l + "mlp.down"] = layer.mlp.up, layer.mlp.down
        return out

    def unused_tensors(self):
        """Names a checkpoint may hold that nothing reads: the norms and convolution of a feed-forward that a layer does not have."""
        return {"l%d.%s" % (i, n) for i, layer in enumerate(self.model.layers) if layer.mlp is None for n in ("norm2", "norm2b", "canon2")}
