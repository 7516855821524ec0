"""The serving engine's host side without a GPU: registry, configuration, padding, cache bookkeeping, batch layout, scheduling and
sampling.  A stand-in model keeps its tokens in the paged pool and its running sum in the state slot, so that a wrong page, slot or
position changes what it generates."""
import json
import subprocess
import sys

import numpy as np
import pytest
import torch

from omniserve_amd import models
from omniserve_amd.engine import Engine, SamplingParams, SequenceInput
from omniserve_amd.engine.cache import Cache, OutOfPages
from omniserve_amd.engine.sampling import filtered_probabilities
from omniserve_amd.models import bobavik, layers
from omniserve_amd.models.base import EngineModel
from omniserve_amd.rope import inverse_frequencies
from oracle import hybrid
from tests.hybrid_util import attention, config, lightning, moe, random_state, tensors

CPU = torch.device("cpu")


class Pages(EngineModel):
    """Next token = hash of the last `span` tokens (read back through the block table) and of the state's sum of all tokens."""
    vocab, dtype, device = 97, torch.float32, CPU

    def __init__(self, span=None):
        self.span = span

    def kv_shapes(self):
        return [(1, 1, 1)]

    def state_shapes(self):
        return [(1, 1, 1)]

    def window(self):
        return self.span

    def linear_workgroups(self):
        return 4

    @staticmethod
    def rule(tokens, span):
        last = tokens[-span:] if span else tokens
        return (sum((i + 1) * t for i, t in enumerate(last)) + 5 * sum(tokens)) % 97

    def forward(self, b, cache):
        pool, state = cache.kv[0][0].view(-1), cache.state[0].view(-1)
        pool[b.kv_slot.long()] = b.tokens.float()
        total = {}

        def answer(t, row):
            n = int(b.pos[t]) + 1
            lo = max(0, n - self.span) if self.span else 0
            at = torch.arange(lo, n)
            page = b.block_table[row].long()[at // 64]
            last = pool[page * 64 + at % 64].long().tolist()
            return (sum((i + 1) * v for i, v in enumerate(last)) + 5 * total[t]) % 97

        rows = {}
        covered = 0
        for first, n, slot, fresh, idx, nseg, *_ in b.segments.tolist():
            s = 0 if idx == 0 and fresh else int(state[slot])
            for t in range(first, first + n):
                s += int(b.tokens[t])
                total[t] = s
            state[slot] = s
            covered += n
        assert covered == b.n_prompt
        for k, (first, n, pos, row) in enumerate(b.entry.tolist()):
            assert [r for e, r in b.attn_tiles.tolist() if e == k] == list(range(0, n, 128))
            assert b.pos[first:first + n].tolist() == list(range(pos, pos + n))
            rows.update({t: row for t in range(first, first + n)})
        for i in range(b.n_decode):
            t = b.n_prompt + i
            slot = int(b.state_slot[i])
            total[t] = (int(state[slot]) if int(b.pos[t]) else 0) + int(b.tokens[t])
            state[slot] = total[t]
            rows[t] = b.n_entries + i
        if not b.rows.numel():
            return None
        z = torch.zeros((b.rows.numel(), self.vocab))
        for r, t in enumerate(b.rows.tolist()):
            z[r, answer(t, rows[t])] = 1.0
        return z

    def greedy(self, z):
        return z.argmax(dim=1)

    def expected(self, prompt, n):
        toks = list(prompt)
        for _ in range(n):
            toks.append(self.rule(toks, self.span))
        return toks[len(prompt):]


def engine(span=None, **kw):
    return Engine(Pages(span), use_graphs=False, **kw)


@pytest.mark.parametrize("span", [None, 1, 64, 65, 150])
@pytest.mark.parametrize("budget", [8, 64, 1000])
def test_scheduler_serves_unequal_requests_from_few_pages(span, budget):
    rng = np.random.default_rng(0)
    e = engine(span, max_tokens=64 * 8, max_seqs=4, max_batch_tokens=budget)
    prompts = [rng.integers(0, 97, n).tolist() for n in (1, 300, 64, 65, 2, 17, 128, 250, 3)]
    gens = [int(n) for n in rng.integers(1, 140, len(prompts))]
    outs = e.generate(prompts, [SamplingParams(max_tokens=n) for n in gens])
    for p, n, o in zip(prompts, gens, outs):
        assert o.tokens == e.model.expected(p, n), len(p)
    assert e.cache.free_pages() == 8 and e.cache.free_slots() == 4


def test_requests_are_put_back_when_pages_run_out():
    e = engine(None, max_tokens=64 * 4, max_seqs=4, max_batch_tokens=512)
    put_back = []
    original = e.scheduler._put_back
    e.scheduler._put_back = lambda r: (put_back.append(r.id), original(r))
    prompts = [[7 * i + j for j in range(40)] for i in range(4)]
    prompts = [[t % 97 for t in p] for p in prompts]
    outs = e.generate(prompts, SamplingParams(max_tokens=100))
    assert put_back and all(o.tokens == e.model.expected(p, 100) for p, o in zip(prompts, outs))


def test_a_request_larger_than_the_cache_is_an_error():
    e = engine(None, max_tokens=64, max_seqs=2, max_batch_tokens=512)
    with pytest.raises(RuntimeError, match="does not fit"):
        e.generate([[1] * 100], SamplingParams(max_tokens=1))


def test_sequences_of_the_caller_may_leave_no_room():
    e = engine(None, max_tokens=256, max_seqs=1)
    s = e.open()
    with pytest.raises(RuntimeError, match="no request can start"):
        e.generate([[1]])
    e.close(s)
    while e.has_work():
        e.step()


def test_stop_tokens_abort_and_bad_requests():
    e = engine(None, max_tokens=1024, max_seqs=2)
    first = e.model.expected([3, 4], 1)[0]
    o = e.generate([[3, 4]], SamplingParams(max_tokens=50, stop_token_ids=(first,)))[0]
    assert o.tokens == [first] and o.finish_reason == "stop"
    a, b = e.add_request([1], SamplingParams(max_tokens=30)), e.add_request([2], SamplingParams(max_tokens=3))
    e.step()
    assert e.abort(a) and not e.abort("nobody")
    done = []
    while e.has_work():
        done += e.step()
    assert [d.id for d in done] == [b] and e.cache.free_slots() == 2
    for bad in ([], [97], [-1]):
        with pytest.raises(ValueError):
            e.add_request(bad)
    s = e.open()
    for x in (SequenceInput(s, []), SequenceInput(s, [97]), SequenceInput(s, [1], [1])):
        with pytest.raises(ValueError):
            e.run([x])
    with pytest.raises(ValueError):
        e.run([SequenceInput(s, [1]), SequenceInput(s, [2])])


def test_cache_pages_and_slots():
    c = Cache(Pages(100), 5, 2, CPU)
    a, b = c.open(), c.open()
    with pytest.raises(RuntimeError):
        c.open()
    c.reserve(a, 130)
    assert a.pages == 3 and c.free_pages() == 2
    c.advance(a, 130)                      # the next token sees from 31 on: page 0 stays
    assert a.released == 0
    c.reserve(a, 33)
    c.advance(a, 33)                       # length 163: sees from 64 on
    assert a.released == 1 and a.table[0] == -1 and c.free_pages() == 3
    c.reserve(b, 192)
    with pytest.raises(OutOfPages):
        c.reserve(a, 64)
    slot = a.slot
    c.close(a)
    assert c.free_pages() == 2 and c.open().slot == slot
    c.close(b)
    assert c.free_pages() == 5


def test_registry_and_config():
    assert "Bobavik" in models.architectures()
    assert models.model_class({"architecture": "Bobavik"}) is bobavik.Bobavik
    with pytest.raises(ValueError):
        models.model_class({"architecture": "Nothing"})
    with pytest.raises(ValueError):
        models.model_class({})
    cfg = config([attention(window=9, rot=16, base=777.0), lightning(mlp=None), attention(v_mix=False, scaling=False, top=1, shared=None)],
                 width=72, vocab=33, eps=1e-3, logit_scale=0.7)
    spec = bobavik.parse_config(json.loads(json.dumps(cfg)))
    assert (spec.width, spec.vocab, spec.eps, spec.logit_scale, spec.norm) == (72, 33, 1e-3, 0.7, "layer")
    a, b, c = (l.mixer for l in spec.layers)
    assert (a.window, a.rotary.dims, a.rotary.base, a.value_mix, a.rotary.scaling["factor"]) == (9, 16, 777.0, True, 8.0)
    assert b.decay == (0.55, 0.93, 0.9985) and spec.layers[1].ff is None
    assert not c.value_mix and c.rotary.scaling is None and spec.layers[2].ff == layers.MoeSpec(6, 1, 48, None)
    for bad in (dict(attention(), type="other"), dict(attention(), mlp={"kind": "dense"}), lightning(decay=[0.5, 1.5, 0.1]), lightning(decay=[0.5, 0.2]),
                attention(heads=3, kv_heads=2), attention(scale=-1.0), attention(window=0), attention(rot=50)):
        with pytest.raises(ValueError):
            bobavik.parse_config(config([bad]))


def test_padding_keeps_the_products():
    g = torch.Generator().manual_seed(1)
    w, x = torch.randn((3 * 40, 72), generator=g), torch.randn((5, 72), generator=g)
    p = layers.pad_out_heads(w, 3, 40, 128)
    y = layers.padded(x, 5, 128) @ p.t()
    assert p.shape == (192, 128)
    assert torch.allclose(y.view(5, 3, 64)[..., :40].reshape(5, 120), x @ w.t(), atol=1e-5) and not y.view(5, 3, 64)[..., 40:].any()
    o = torch.randn((72, 120), generator=g)
    back = y @ layers.pad_in_heads(o, 3, 40, 128).t()
    assert torch.allclose(back[:, :72], x @ w.t() @ o.t(), atol=1e-3) and not back[:, 72:].any()
    gate, up = torch.arange(40.)[:, None].expand(40, 8), 100 + torch.arange(40.)[:, None].expand(40, 8)
    r = layers.pair_rows(gate, up, 64, 8)
    assert r[:16, 0].tolist() == list(range(16)) and r[16:32, 0].tolist() == list(range(100, 116)) and r[32, 0] == 16
    assert r[64:72, 0].tolist() == list(range(32, 40)) and not r[72:80].any()
    assert [layers.pad_head(n) for n in (1, 64, 65, 128, 129, 256)] == [64, 64, 128, 128, 256, 256]
    with pytest.raises(ValueError):
        layers.pad_head(257)


@pytest.mark.parametrize("scaling", [None, dict(factor=8.0, low=1.0, high=4.0, original=200), dict(factor=2.0, low=2.0, high=3.0, original=50)])
def test_rotary_frequencies(scaling):
    a, b = inverse_frequencies(48, 5000.0, scaling), hybrid.rope_frequencies(48, 5000.0, scaling)
    assert np.allclose(a, b, rtol=1e-14) and len(a) == 24
    if scaling:
        plain = hybrid.rope_frequencies(48, 5000.0)
        kinds = {"kept": (b == plain).any(), "divided": np.isclose(b, plain / scaling["factor"], rtol=1e-12).any()}
        assert all(kinds.values()), kinds


def test_weights_report_missing_misshapen_and_unused():
    cfg = config([attention(), lightning()])
    state = random_state(cfg)
    w = layers.Weights(state, CPU, torch.float32)
    assert w.under("l0.").under("mix.").matrix("q", 4 * 48, 160).dtype == torch.float32
    assert w.vector("final.norm", 160, 192).shape == (192,)
    assert 0 < w.under("l0.mix.").scalar("vmix") < 1
    with pytest.raises(RuntimeError, match="lacks"):
        w.matrix("nothing", 1, 1)
    with pytest.raises(RuntimeError, match="shape"):
        w.matrix("embed", 1, 1)
    left = w.leftovers(optional=(".mix.vmix",))
    assert "embed" in left and "l0.mix.q" not in left and set(left) < set(tensors(cfg))


def test_oracle_recurrence_and_window_by_hand():
    q = k = np.array([[[1.0]], [[2.0]], [[3.0]]])
    v = np.array([[[1.0]], [[1.0]], [[2.0]]])
    o, s = hybrid.decayed_linear_attention(q, k, v, [0.5])
    assert o[:, 0, 0].tolist() == [1.0, 2 * (0.5 + 2), 3 * (0.25 + 1 + 6)] and s[0, 0, 0] == 7.25
    a = hybrid.windowed_attention(np.zeros((4, 1, 1)), np.zeros((4, 1, 1)), np.arange(4.0).reshape(4, 1, 1), 1.0, 2)
    assert a[:, 0, 0].tolist() == [0.0, 0.5, 1.5, 2.5]
    ids, w = hybrid.route(np.array([[0.0, 3.0, 3.0, 1.0]]), np.eye(4), np.zeros(4), 2)
    assert ids.tolist() == [[1, 2]] and w.tolist() == [[0.5, 0.5]]


def test_sampling_filters():
    z = torch.log(torch.tensor([0.5, 0.3, 0.15, 0.05]))
    p = filtered_probabilities(z, SamplingParams(temperature=1.0))
    assert torch.allclose(p, torch.tensor([0.5, 0.3, 0.15, 0.05]), atol=1e-6)
    assert filtered_probabilities(z, SamplingParams(temperature=1.0, top_k=2)).tolist() == pytest.approx([0.625, 0.375, 0, 0])
    assert filtered_probabilities(z, SamplingParams(temperature=1.0, top_p=0.6)).tolist() == pytest.approx([0.625, 0.375, 0, 0])
    assert filtered_probabilities(z, SamplingParams(temperature=1.0, top_p=1e-6)).tolist() == [1, 0, 0, 0]
    assert filtered_probabilities(z, SamplingParams(temperature=0.5)).tolist() == pytest.approx((p * p / (p * p).sum()).tolist())
    for bad in (dict(temperature=-1), dict(top_p=0), dict(max_tokens=0), dict(top_k=-1)):
        with pytest.raises(ValueError):
            SamplingParams(**bad)
    e = engine(None, max_tokens=256, max_seqs=2)
    a = [o.tokens for o in e.generate([[1, 2]] * 2, SamplingParams(max_tokens=8, temperature=5.0, seed=3))]
    b = [o.tokens for o in e.generate([[1, 2]] * 2, SamplingParams(max_tokens=8, temperature=5.0, seed=3))]
    assert a == b and a[0] == a[1]


def test_trace_replay_rejects_what_it_cannot_run(tmp_path):
    import os
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Nothing"}))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32", "--out",
                        str(tmp_path), "--max-tokens", "64"], input="", text=True, capture_output=True, timeout=100)
    assert r.returncode not in (0, 3) and "unknown architecture" in r.stderr


def test_command_line(tmp_path, capsys):
    from omniserve_amd import cli
    assert cli.main(["models"]) == 0
    assert {"Bobavik", "LlamaForCausalLM"} <= set(capsys.readouterr().out.split())
    a = cli.parser().parse_args(["generate", "--model", "m", "--prompt-ids", "1, 2,3", "--prompt-ids", "4", "--stop-ids", "7,8"])
    assert a.prompt_ids == [[1, 2, 3], [4]] and a.stop_ids == [7, 8] and a.temperature == 0
    assert cli.main(["generate", "--model", str(tmp_path)]) == 2
    with pytest.raises(SystemExit):
        cli.main(["generate", "--model", "m", "--prompt-ids", "x"])
    with pytest.raises(SystemExit):
        cli.main(["trace", "--nothing"])


def test_llama_config():
    from omniserve_amd.models import qserve_llama
    c = qserve_llama.parse_config({"hidden_size": 512, "intermediate_size": 1024, "num_attention_heads": 4, "num_key_value_heads": 2,
                                   "num_hidden_layers": 3, "vocab_size": 99, "rope_theta": 5e5, "quantization": {"group_size": 128}})
    assert (c.head_dim, c.kv_heads, c.layers, c.group_size, c.rope_theta) == (128, 2, 3, 128, 5e5)
    assert models.model_class({"architectures": ["LlamaForCausalLM"]}) is qserve_llama.QServeLlama
