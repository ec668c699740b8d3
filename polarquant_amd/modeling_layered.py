"""The shell of models whose layers keep their sequences' state in arenas: cache tuples, left padding, portions, logits.

An arena is what one layer run keeps of B sequences.  It has `kv_len` (tokens so far), `start` (left padding, int32 [B] or
None), `reserve(tokens)`, `reset()`, `as_tuple()` (a `PolarCache`: the state's tensors, then kv_len), `load(parts, n)` (the
tensors of such a tuple, copied in) and `step_state()` (tensors that running a step twice would change twice).

The forward takes prompts, portions of prompts of any length, and single tokens alike.
"""
from __future__ import annotations

from typing import List, Optional

import torch
import torch.nn as nn

from . import layer_ops as ops
from .modeling_common import PolarForCausalLM, CausalLMOutputWithPast


class LayeredModel(nn.Module):
    """Embedding and `build_layers(config)`; `capture`, if a list, receives the residual stream after every layer run."""

    def __init__(self, config):
        super().__init__()
        self.config = config
        self.embed_tokens = nn.Embedding(config.vocab_size, config.hidden_size)
        self.layers = nn.ModuleList(self.build_layers(config))
        self.capture: Optional[List[torch.Tensor]] = None

    def build_layers(self, config):
        raise NotImplementedError

    def new_arenas(self, B: int, capacity: int) -> List:
        """One arena per layer run, for B sequences of `capacity` tokens to begin with."""
        raise NotImplementedError

    def run(self, input_ids: torch.Tensor, arenas: List, pos: int, pos_dev: Optional[torch.Tensor] = None, plan=None) -> torch.Tensor:
        """The layers over tokens [B, L] at positions pos .. (or *pos_dev .., with a `plan` of step_plan): appends to the
        arenas' tensors and returns the normed hidden states; the arenas' host counts are the caller's to advance."""
        raise NotImplementedError

    def step_plan(self, B: int, max_len: int, device):
        """What `run` needs to know ahead to run one token at a position it learns from the device."""
        return None

    # -- cache plumbing
    def _arenas_of(self, past_key_values, B: int) -> List:
        arenas = [getattr(t, "arena", None) for t in past_key_values]
        if all(a is not None for a in arenas):
            if any(a.kv_len != t[-1] for a, t in zip(arenas, past_key_values)):
                raise ValueError("polarquant_amd: a cache of %d tokens was handed in whose state has moved on to %d (a running "
                                 "state exists for the newest token only)" % (past_key_values[0][-1], arenas[0].kv_len))
            return arenas
        n = past_key_values[0][-1]                # plain tuples: copy them into fresh arenas
        arenas = self.new_arenas(B, (self.config.cache_capacity or n + 1024))
        for a, t in zip(arenas, past_key_values):
            a.load(t[:-1], n)
        return arenas

    @staticmethod
    def _left_padding(mask: Optional[torch.Tensor]) -> Optional[torch.Tensor]:
        """int32 [B] count of leading zeros of the mask [B, L], None if there are none."""
        if mask is None:
            return None
        m = mask != 0
        if bool(m.all()):
            return None
        if bool((m[:, 1:] < m[:, :-1]).any()):
            raise ValueError("polarquant_amd: the attention mask may only mark left padding (zeros in front of ones)")
        return (~m).sum(1).to(torch.int32)

    @torch.no_grad()
    def forward(self, input_ids=None, attention_mask=None, past_key_values=None):
        """-> (normed hidden states [B, L, W], tuple of per-layer cache tuples).  Any number of new tokens, with or without
        a cache.  attention_mask [B, tokens so far] may mark left padding; it is read with the first tokens of a sequence."""
        B, L = input_ids.shape
        if past_key_values is None:
            arenas, n = self.new_arenas(B, self.config.cache_capacity or L + 1024), 0
        else:
            arenas, n = self._arenas_of(past_key_values, B), past_key_values[0][-1]
        if n == 0:
            start = self._left_padding(attention_mask)
            for a in arenas:
                a.start = start
        for a in arenas:
            a.reserve(n + L)
        h = self.run(input_ids, arenas, n)
        for a in arenas:
            a.kv_len = n + L
        return h, tuple(a.as_tuple() for a in arenas)


class LayeredForCausalLM(PolarForCausalLM):
    """The framework's causal-LM shell over a `LayeredModel`; logits are float32."""

    model_class = LayeredModel

    def forward(self, input_ids=None, attention_mask=None, past_key_values=None, num_logits_to_keep=0, return_dict=True,
                logit_positions: Optional[torch.Tensor] = None):
        """logit_positions: indices into the new tokens whose logits are wanted, instead of the last num_logits_to_keep."""
        h, past = self.model(input_ids=input_ids, attention_mask=attention_mask, past_key_values=past_key_values)
        h = h[:, -num_logits_to_keep:] if logit_positions is None else h.index_select(1, logit_positions)
        return CausalLMOutputWithPast(logits=self.logits(h), past_key_values=past)

    @torch.no_grad()
    def logits(self, h: torch.Tensor) -> torch.Tensor:
        return ops.linear_f32(h.contiguous(), self.lm_head.weight)

    def new_cache(self, batch: int, capacity: int):
        """An empty cache of `capacity` tokens per sequence, to hand in as past_key_values."""
        return tuple(a.as_tuple() for a in self.model.new_arenas(batch, capacity))

    @staticmethod
    def reset_cache(past_key_values):
        """The cache's memory as an empty cache."""
        for t in past_key_values:
            t.arena.reset()
        return tuple(t.arena.as_tuple() for t in past_key_values)

    def graph_decoder(self, max_len: int):
        from .graph_decode import LayeredGraphDecoder
        return LayeredGraphDecoder(self, max_len)
