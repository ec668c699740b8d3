"""The Kapudra decoder through the framework's own entry points, against the plain float64 implementation."""
import io
import json
import os

import pytest
import torch

from oracle import kapudra_oracle as ko
from polarquant_amd.checkpoint import load_generation_config, load_pretrained
from polarquant_amd.graph_decode import LayeredGraphDecoder
from polarquant_amd.modeling_common import GenerationConfig, generate

import kapudra_cases as kc

pytestmark = pytest.mark.gpu
LIMIT = {torch.float32: 1e-4, torch.bfloat16: 8e-2, torch.float16: 1.2e-2}        # worst row, relative root mean square


def load(tmp_path, name, seed, dtype, gpu, cfg=None, w=None):
    cfg = cfg or kc.ALL[name]
    path = str(tmp_path / ("m%d" % seed))
    w = kc.write(path, cfg, seed, kc.RANKS[name], w)
    return load_pretrained(path, dtype, gpu), cfg, w


def feed(model, toks, cuts, past=None):
    """Logits of `toks` run in portions of the given sizes."""
    out, at = [], 0
    for n in cuts:
        r = model(input_ids=torch.tensor([toks[at:at + n]], device=model.device), past_key_values=past)
        past = r.past_key_values
        out.append(r.logits[0])
        at += n
    assert at == len(toks)
    return torch.cat(out), past


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16, torch.float16])
@pytest.mark.parametrize("name", sorted(kc.ALL))
def test_prompts_and_layers(gpu, tmp_path, name, dtype):
    model, cfg, w = load(tmp_path, name, 11, dtype, gpu)
    for n in (1, 2, 17, 65, 150):
        t = kc.tokens(n, cfg["vocab"], n)
        cap = []
        want = ko.forward(t, cfg, w, capture=cap)
        model.model.capture = []
        got = feed(model, t, [n])[0]
        assert got.dtype == torch.float32
        for i, (a, b) in enumerate(zip(model.model.capture, cap)):
            assert kc.close(a[0], b, LIMIT[dtype]), (n, "layer run", i)
        assert len(model.model.capture) == len(cap)
        model.model.capture = None
        assert kc.close(got, want, LIMIT[dtype]), n


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", sorted(kc.ALL))
def test_portions_and_token_by_token(gpu, tmp_path, name, dtype):
    """Whole, in portions down to two tokens with edges around every tile, strip and chunk, and one by one."""
    model, cfg, w = load(tmp_path, name, 12, dtype, gpu)
    n = 211
    t = kc.tokens(n, cfg["vocab"], 5)
    want = ko.forward(t, cfg, w)
    for cuts in ([n], [1] * n, [2] * 105 + [1], [16, 17, 32, 33, 43, 70], [63, 1, 64, 83], [64, 64, 83], [65, 63, 2, 81], [3, 2, 1, 205], [127, 1, 1, 82], [40, 130, 41]):
        assert kc.close(feed(model, t, cuts)[0], want, LIMIT[dtype]), cuts


def test_memory_of_ended_sequences_is_used_again(gpu, tmp_path):
    for name, dtype in (("even", torch.bfloat16), ("odd", torch.float32)):
        model, cfg, w = load(tmp_path, name, 14, dtype, gpu)
        past = model.new_cache(1, 192)
        for n, seed in ((180, 1), (3, 2), (70, 3), (1, 4), (150, 5)):
            t = kc.tokens(n, cfg["vocab"], seed)
            cuts = [n] if n < 100 else [n - 40, 2] + [1] * 38
            got, past = feed(model, t, cuts, past)
            assert kc.close(got, ko.forward(t, cfg, w), LIMIT[dtype]), (name, n)
            states = [s for p in past for s in p.arena.states]
            address = [s.tensors()[-1].data_ptr() for s in states]
            past = model.reset_cache(past)
            assert past[0][-1] == 0 and address == [s.tensors()[-1].data_ptr() for s in states]
            for s in states:
                if hasattr(s, "k"):
                    s.k.fill_(100.0), s.v.fill_(100.0)              # whatever is left behind must not matter


def test_tuples_are_guarded_and_copied(gpu, tmp_path):
    model, cfg, w = load(tmp_path, "even", 15, torch.float32, gpu)
    t = kc.tokens(90, cfg["vocab"], 1)
    want = ko.forward(t, cfg, w)
    got, past = feed(model, t[:40], [40], model.new_cache(1, 10))
    more, past2 = feed(model, t[40:], [20, 1, 29], past)
    assert kc.close(torch.cat([got, more]), want, LIMIT[torch.float32])
    with pytest.raises(ValueError, match="moved on"):
        feed(model, t[40:], [50], past)
    plain = tuple(tuple(x.clone() if torch.is_tensor(x) else x for x in p) for p in past2)
    nxt = kc.tokens(5, cfg["vocab"], 2)
    assert kc.close(feed(model, nxt, [5], plain)[0], ko.forward(t + nxt, cfg, w)[-5:], LIMIT[torch.float32])


def test_passes_have_states_of_their_own(gpu, tmp_path):
    model, cfg, _ = load(tmp_path, "even", 16, torch.bfloat16, gpu)
    past = model.new_cache(2, 1)
    assert len(past) == len(ko.schedule(cfg)) == 1 + 2 * 3 + 1
    tensors = [x for p in past for s in p.arena.states for x in s.tensors()]
    assert len({x.data_ptr() for x in tensors}) == len(tensors)
    assert model.state_bytes() * 2 == sum(x.numel() * x.element_size() for x in tensors)


@pytest.mark.parametrize("name,dtype", [("even", torch.bfloat16), ("odd", torch.float32), ("wide", torch.float16), ("ones", torch.bfloat16)])
def test_batch_of_unequal_prompts(gpu, tmp_path, name, dtype):
    """Left-padded prompts decoded together, each against itself alone."""
    model, cfg, w = load(tmp_path, name, 16, dtype, gpu)
    lens, L, new = [70, 1, 33, 69], 70, 6
    seqs = [kc.tokens(n + new, cfg["vocab"], 20 + n) for n in lens]
    ids = torch.zeros(4, L, dtype=torch.long)
    mask = torch.zeros(4, L, dtype=torch.long)
    for b, (n, s) in enumerate(zip(lens, seqs)):
        ids[b, L - n:], mask[b, L - n:] = torch.tensor(s[:n]), 1
    out = model(input_ids=ids.to(gpu), attention_mask=mask.to(gpu))
    logits = [out.logits[b, L - n:] for b, n in enumerate(lens)]
    for i in range(new):
        mask = torch.cat([mask, torch.ones(4, 1, dtype=torch.long)], 1)
        out = model(input_ids=torch.tensor([[s[n + i]] for n, s in zip(lens, seqs)], device=gpu), attention_mask=mask.to(gpu), past_key_values=out.past_key_values)
        logits = [torch.cat([a, out.logits[b]]) for b, a in enumerate(logits)]
    for b, s in enumerate(seqs):
        assert kc.close(logits[b], ko.forward(s, cfg, w), LIMIT[dtype]), b


def test_long_decoding(gpu, tmp_path):
    for name, dtype in (("even", torch.bfloat16), ("wide", torch.float32)):
        model, cfg, w = load(tmp_path, name, 17, dtype, gpu)
        t = kc.tokens(420, cfg["vocab"], 3)
        assert kc.close(feed(model, t, [20] + [1] * 400)[0], ko.forward(t, cfg, w), LIMIT[dtype])


def test_graph_replays_equal_the_eager_step(gpu, tmp_path):
    for name, dtype in (("even", torch.bfloat16), ("odd", torch.float32), ("wide", torch.float16)):
        model, cfg, w = load(tmp_path, name, 18, dtype, gpu)
        B, L, new = 3, 50, 24
        ids = torch.tensor([kc.tokens(L, cfg["vocab"], b) for b in range(B)], device=gpu)
        feed_ids = torch.tensor([kc.tokens(new, cfg["vocab"], 50 + b) for b in range(B)], device=gpu)
        mask = torch.ones(B, L, dtype=torch.long, device=gpu)
        mask[1, :7] = 0
        runs = []
        for use_graph in (True, False):
            dec = LayeredGraphDecoder(model, L + new + 1, use_graph=use_graph)
            got = [dec.prefill(ids, mask)]
            for i in range(new):
                got.append(dec.step(feed_ids[:, i:i + 1]).clone())
                if i % 5 == 0:                                  # the program's own work between replays
                    torch.cuda.synchronize()
                    _ = (got[-1] * 2).sum().item()
            runs.append(torch.cat(got, 1))
            assert dec.cache()[0][-1] == L + new
        assert torch.equal(runs[0], runs[1]), name
        out = model(input_ids=ids, attention_mask=mask, num_logits_to_keep=1)
        eager = [out.logits]
        for i in range(new):
            out = model(input_ids=feed_ids[:, i:i + 1], past_key_values=out.past_key_values)
            eager.append(out.logits)
        assert kc.rel_rms(runs[0].flatten(0, 1), torch.cat(eager, 1).flatten(0, 1).cpu()) < (LIMIT[torch.float32] if dtype == torch.float32 else 2e-2)
        for b in range(B):
            s = (7 if b == 1 else 0)
            want = ko.forward(ids[b, s:].tolist() + feed_ids[b].tolist(), cfg, w)[-new - 1:]
            assert kc.close(runs[0][b], want, LIMIT[dtype]), (name, b)


def _greedy(cfg, w, prompt, n):
    out = []
    for _ in range(n):
        out.append(int(ko.forward(prompt + out, cfg, w)[-1].argmax()))
    return out


def test_greedy_generation(gpu, tmp_path):
    """generate(): eager and graph-replayed, one sequence and a left-padded batch, against the oracle's own greedy loop."""
    model, cfg, w = load(tmp_path, "even", 19, torch.float32, gpu)
    prompts = [kc.tokens(n, cfg["vocab"], n) for n in (40, 23)]
    want = [_greedy(cfg, w, p, 12) for p in prompts]
    gc = GenerationConfig(eos_token_id=[cfg["vocab"] + 1])
    for graph in (False, True):
        one = generate(model, torch.tensor([prompts[0]], device=gpu), None, gc, max_new_tokens=12, graph_decoder=graph)
        assert one[0].tolist() == want[0], graph
        ids = torch.tensor([prompts[0], [0] * 17 + prompts[1]], device=gpu)
        mask = torch.ones_like(ids)
        mask[1, :17] = 0
        two = generate(model, ids, mask, gc, max_new_tokens=12, graph_decoder=graph)
        assert two.tolist() == want, graph
    stop = GenerationConfig(eos_token_id=[want[0][4]])
    first = want[0].index(want[0][4])
    assert generate(model, torch.tensor([prompts[0]], device=gpu), None, stop, max_new_tokens=12)[0].tolist() == want[0][:first + 1]
    torch.manual_seed(0)
    top1 = GenerationConfig(eos_token_id=[cfg["vocab"] + 1], top_k=1)
    assert generate(model, torch.tensor([prompts[0]], device=gpu), None, top1, do_sample=True, max_new_tokens=12)[0].tolist() == want[0]


def test_trace_replay(gpu, tmp_path, monkeypatch, capsys):
    from polarquant_amd import trace_replay
    import numpy as np
    cfg = kc.ODD
    w = kc.write(str(tmp_path / "m"), cfg, 21, kc.RANKS["odd"])
    t = {n: kc.tokens(k, cfg["vocab"], k) for n, k in (("a", 30), ("b", 9))}
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": t["a"][:20], "want": [3, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": t["a"][20:22], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": t["a"][22:], "want": [0, 7]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": t["b"], "want": [8]}], "end": ["b"]}]
    for dtype, limit in (("float32", 1e-4), ("bfloat16", 8e-2)):
        out = tmp_path / dtype
        out.mkdir()
        monkeypatch.setattr("sys.stdin", io.StringIO("".join(json.dumps(s) + "\n" for s in steps)))
        assert trace_replay.main(["--model", str(tmp_path / "m"), "--dtype", dtype, "--out", str(out), "--max-tokens", "30"]) == 0
        assert capsys.readouterr().out.split("\n")[:4] == ["done 0", "done 1", "done 2", "done 3"]
        assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "3.f32"]
        read = lambda s: torch.from_numpy(np.fromfile(str(out / ("%d.f32" % s)), dtype="<f4")).view(-1, cfg["vocab"])
        a, b = ko.forward(t["a"], cfg, w), ko.forward(t["b"], cfg, w)
        for s, want in ((0, a[[3, 19]]), (2, a[[22, 29]]), (3, b[[8]])):
            assert kc.close(read(s), want, limit)
    with pytest.raises(ValueError, match="vocabulary"):
        monkeypatch.setattr("sys.stdin", io.StringIO(json.dumps({"step": 0, "entries": [{"id": "x", "tokens": [cfg["vocab"]], "want": []}], "end": []})))
        trace_replay.main(["--model", str(tmp_path / "m"), "--out", str(tmp_path)])


def test_command_line(gpu, tmp_path, monkeypatch):
    """The evaluation command line serves the design from its checkpoint directory (a byte tokenizer stands in)."""
    import sys
    import types
    from polarquant_amd import accuracy_eval

    class Bytes:
        def encode(self, s):
            return [b % 256 for b in s.encode()][-60:]

        def batch_decode(self, ids, skip_special_tokens=True):
            return [" ".join(str(int(i)) for i in row) for row in ids]

    monkeypatch.setitem(sys.modules, "transformers", types.SimpleNamespace(AutoTokenizer=types.SimpleNamespace(from_pretrained=lambda *a, **k: Bytes())))
    cfg = dict(kc.EVEN, eos_token_id=7)
    kc.write(str(tmp_path / "m"), cfg, 22)
    assert load_generation_config(str(tmp_path / "m")).eos_token_id == [7]
    data = tmp_path / "q.jsonl"
    data.write_text(json.dumps({"conversations": [{"value": "What is 1 + 1?"}, {"value": "The answer is 2"}]}) + "\n")
    rows = []
    for extra in ([], ["--graph"]):
        accuracy_eval.main(["gsm8k", "--model", str(tmp_path / "m"), "--data", str(data), "--out", str(tmp_path / "o.jsonl"), "--chat", "none"] + extra)
        rows.append(json.loads((tmp_path / "o.jsonl").read_text()))
    assert rows[0]["output_text"] and len(rows[0]["output_text"].split()) == len(rows[1]["output_text"].split()) or 7 in map(int, rows[0]["output_text"].split())
