"""The Dekipel decoder through the framework's own entry points, against the plain float64 implementation."""
import io
import json
import os

import pytest
import torch

from oracle import dekipel_oracle as do
from polarquant_amd.checkpoint import load_generation_config, load_pretrained
from polarquant_amd.graph_decode import LayeredGraphDecoder
from polarquant_amd.modeling_common import GenerationConfig, generate

import dekipel_cases as dc

pytestmark = pytest.mark.gpu
LIMIT = {torch.float32: 2e-5, torch.bfloat16: 6e-2, torch.float16: 9e-3}        # worst row, relative root mean square


def load(tmp_path, cfg, seed, dtype, gpu, weights=None):
    w = dc.write(str(tmp_path / ("m%d" % seed)), cfg, seed, weights=weights)
    return load_pretrained(str(tmp_path / ("m%d" % seed)), dtype, gpu), w


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
@pytest.mark.parametrize("name", sorted(dc.ALL))
def test_prompts_and_layers(gpu, tmp_path, name, dtype):
    cfg = dc.ALL[name]
    model, w = load(tmp_path, cfg, 11, dtype, gpu)
    for n in (1, 2, 17, 65, 150):
        t = dc.tokens(n, cfg["vocab"], n)
        cap = []
        want = do.forward(t, cfg, w, capture=cap)
        model.model.capture = []
        got = feed(model, t, [n])[0]
        assert got.dtype == torch.float32
        for i, (a, b) in enumerate(zip(model.model.capture, cap)):
            assert dc.rel_rms(a[0], b) < LIMIT[dtype], (n, "layer", i)
        assert len(model.model.capture) == len(cap)
        model.model.capture = None
        assert dc.rel_rms(got, want) < LIMIT[dtype], n


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", sorted(dc.ALL))
def test_portions_and_token_by_token(gpu, tmp_path, name, dtype):
    """Whole, in portions down to two tokens with edges around every tile and strip, and one by one."""
    cfg = dc.ALL[name]
    model, w = load(tmp_path, cfg, 12, dtype, gpu)
    n = 141
    t = dc.tokens(n, cfg["vocab"], 5)
    want = do.forward(t, cfg, w)
    for cuts in ([n], [1] * n, [2] * 70 + [1], [16, 17, 32, 33, 43], [63, 1, 64, 13], [64, 64, 13], [65, 63, 2, 11], [3, 2, 1, 135], [127, 1, 1, 12]):
        assert dc.rel_rms(feed(model, t, cuts)[0], want) < LIMIT[dtype], cuts


def test_far_keys_and_sinks_show(gpu, tmp_path):
    """Sharp attention: with the scores scaled up a single far key carries most of the weight, so that a lost key, a key
    too many or a lost sink changes the logits far beyond the tolerance (which the altered oracle must exceed)."""
    for dtype, sharp, limit in ((torch.float32, 3.0, 5e-5), (torch.bfloat16, 1.5, 7e-2)):     # (16-bit rounding of sharp scores is loud)
        cfg = json.loads(json.dumps(dc.EVEN))
        for l in cfg["layers"]:
            l["mixer"]["scale"] *= sharp
        w = do.random_weights(cfg, 13)
        for i in range(len(cfg["layers"])):
            w["l%d.mix.sink" % i] = torch.linspace(2.0, 9.0, cfg["layers"][i]["mixer"]["heads"]).bfloat16()
        t = dc.tokens(230, cfg["vocab"], 6)
        want = do.forward(t, cfg, w)
        no_sink = do.forward(t, cfg, {k: (v - 1e4 if k.endswith("sink") else v) for k, v in w.items()})
        assert dc.rel_rms(no_sink, want) > 3 * limit
        if dtype == torch.float32:
            assert dc.rel_rms(do.forward(t[1:], cfg, w), want[1:]) > 100 * limit
        model, _ = load(tmp_path, cfg, 13, dtype, gpu, w)
        for cuts in ([230], [100] + [1] * 130, [37, 2, 64, 127]):
            assert dc.rel_rms(feed(model, t, cuts)[0], want) < limit, (dtype, cuts)


def test_memory_of_ended_sequences_is_used_again(gpu, tmp_path):
    for name, dtype in (("even", torch.bfloat16), ("odd", torch.float32)):
        cfg = dc.ALL[name]
        model, w = load(tmp_path, cfg, 14, dtype, gpu)
        past = model.new_cache(1, 192)
        for n, seed in ((180, 1), (3, 2), (70, 3), (1, 4), (150, 5)):
            t = dc.tokens(n, cfg["vocab"], seed)
            cuts = [n] if n < 100 else [n - 40, 2] + [1] * 38
            got, past = feed(model, t, cuts, past)
            assert dc.rel_rms(got, do.forward(t, cfg, w)) < LIMIT[dtype], (name, n)
            address = past[0].arena.c.data_ptr()
            past = model.reset_cache(past)
            assert past[0][-1] == 0 and past[0].arena.c.data_ptr() == address
            for a in (p.arena for p in past):
                if a.source is None:
                    a.c[:, -1:].fill_(100.0)            # whatever is left behind must not matter


def test_cache_grows_and_tuples_are_guarded(gpu, tmp_path):
    cfg = dc.EVEN
    model, w = load(tmp_path, cfg, 15, torch.float32, gpu)
    t = dc.tokens(90, cfg["vocab"], 1)
    want = do.forward(t, cfg, w)
    got, past = feed(model, t[:40], [40], model.new_cache(1, 10))          # 64 rows to begin with
    more, past2 = feed(model, t[40:], [20, 1, 29], past)
    assert dc.rel_rms(torch.cat([got, more]), want) < 2e-5
    with pytest.raises(ValueError, match="moved on"):
        feed(model, t[40:], [50], past)
    # plain tuples (no arena) are copied
    plain = tuple(tuple(x.clone() if torch.is_tensor(x) else x for x in p) for p in past2)
    nxt = dc.tokens(5, cfg["vocab"], 2)
    want = do.forward(t + nxt, cfg, w)[-5:]
    assert dc.rel_rms(feed(model, nxt, [5], plain)[0], want) < 2e-5


@pytest.mark.parametrize("name,dtype", [("even", torch.bfloat16), ("odd", torch.float32), ("padded", torch.float16)])
def test_batch_of_unequal_prompts(gpu, tmp_path, name, dtype):
    """Left-padded prompts decoded together, each against itself alone."""
    cfg = dc.ALL[name]
    model, w = load(tmp_path, cfg, 16, dtype, gpu)
    lens, L, new = [70, 1, 33, 69], 70, 6
    seqs = [dc.tokens(n + new, cfg["vocab"], 20 + n) for n in lens]
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
        assert dc.rel_rms(logits[b], do.forward(s, cfg, w)) < LIMIT[dtype], b


def test_long_decoding(gpu, tmp_path):
    cfg = dc.PADDED
    model, w = load(tmp_path, cfg, 17, torch.bfloat16, gpu)
    t = dc.tokens(420, cfg["vocab"], 3)
    assert dc.rel_rms(feed(model, t, [20] + [1] * 400)[0], do.forward(t, cfg, w)) < LIMIT[torch.bfloat16]


def test_graph_replays_equal_the_eager_step(gpu, tmp_path):
    for name, dtype in (("even", torch.bfloat16), ("odd", torch.float32)):
        cfg = dc.ALL[name]
        model, w = load(tmp_path, cfg, 18, dtype, gpu)
        B, L, new = 3, 50, 24
        ids = torch.tensor([dc.tokens(L, cfg["vocab"], b) for b in range(B)], device=gpu)
        feed_ids = torch.tensor([dc.tokens(new, cfg["vocab"], 50 + b) for b in range(B)], device=gpu)
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
        assert dc.rel_rms(runs[0].flatten(0, 1), torch.cat(eager, 1).flatten(0, 1).cpu()) < (2e-5 if dtype == torch.float32 else 1e-2)
        for b in range(B):
            s = (7 if b == 1 else 0)
            want = do.forward(ids[b, s:].tolist() + feed_ids[b].tolist(), cfg, w)[-new - 1:]
            assert dc.rel_rms(runs[0][b], want) < LIMIT[dtype], (name, b)


def _greedy(cfg, w, prompt, n):
    out = []
    for _ in range(n):
        out.append(int(do.forward(prompt + out, cfg, w)[-1].argmax()))
    return out


def test_greedy_generation(gpu, tmp_path):
    """generate(): eager and graph-replayed, one sequence and a left-padded batch, against the oracle's own greedy loop."""
    cfg = dc.EVEN
    model, w = load(tmp_path, cfg, 19, torch.float32, gpu)
    prompts = [dc.tokens(n, cfg["vocab"], n) for n in (40, 23)]
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
    cfg = dc.ODD
    w = dc.write(str(tmp_path / "m"), cfg, 21)
    t = {n: dc.tokens(k, cfg["vocab"], k) for n, k in (("a", 30), ("b", 9))}
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": t["a"][:20], "want": [3, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": t["a"][20:22], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": t["a"][22:], "want": [0, 7]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": t["b"], "want": [8]}], "end": ["b"]}]
    for dtype, limit in (("float32", 2e-5), ("bfloat16", 5e-2)):
        out = tmp_path / dtype
        out.mkdir()
        monkeypatch.setattr("sys.stdin", io.StringIO("".join(json.dumps(s) + "\n" for s in steps)))
        assert trace_replay.main(["--model", str(tmp_path / "m"), "--dtype", dtype, "--out", str(out), "--max-tokens", "30"]) == 0
        assert capsys.readouterr().out.split("\n")[:4] == ["done 0", "done 1", "done 2", "done 3"]
        assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "3.f32"]
        read = lambda s: torch.from_numpy(np.fromfile(str(out / ("%d.f32" % s)), dtype="<f4")).view(-1, cfg["vocab"])
        a, b = do.forward(t["a"], cfg, w), do.forward(t["b"], cfg, w)
        for s, want in ((0, a[[3, 19]]), (2, a[[22, 29]]), (3, b[[8]])):
            assert dc.rel_rms(read(s), want) < limit
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
    cfg = dict(dc.EVEN, eos_token_id=7)
    dc.write(str(tmp_path / "m"), cfg, 22)
    assert load_generation_config(str(tmp_path / "m")).eos_token_id == [7]
    data = tmp_path / "q.jsonl"
    data.write_text(json.dumps({"conversations": [{"value": "What is 1 + 1?"}, {"value": "The answer is 2"}]}) + "\n")
    rows = []
    for extra in ([], ["--graph"]):
        accuracy_eval.main(["gsm8k", "--model", str(tmp_path / "m"), "--data", str(data), "--out", str(tmp_path / "o.jsonl"), "--chat", "none"] + extra)
        rows.append(json.loads((tmp_path / "o.jsonl").read_text()))
    assert rows[0]["output_text"] and len(rows[0]["output_text"].split()) == len(rows[1]["output_text"].split()) or 7 in map(int, rows[0]["output_text"].split())
