"""The W4A8KV4 Llama on the serving engine against runtime.DecodeRunner with the same checkpoint and prompts."""
import json

import numpy as np
import pytest
import torch

from omniserve_amd import ckpt, models
from omniserve_amd.engine import Engine, SamplingParams, SequenceInput

pytestmark = pytest.mark.gpu
DEV = torch.device("cuda:0")


@pytest.mark.parametrize("group_size", [-1, 128])
def test_generation_equals_the_runner(tmp_path, group_size):
    from omniserve_amd.runtime import DecodeRunner
    _, cfg = ckpt.make_tiny_checkpoint(str(tmp_path), group_size=group_size, seed=3)
    B, L, n = 3, 70, 12
    prompts = np.random.default_rng(1).integers(0, cfg.vocab, (B, L)).tolist()
    r = DecodeRunner(cfg, batch=B, context=L, max_new=n + 2, device=DEV, use_graph=False, fused=1)
    ckpt.load_into_runner(r, ckpt.load_state_dict(str(tmp_path)))
    r.prefill(L, tokens=torch.tensor(prompts, device=DEV).view(-1))
    want = [r.tokens.clone()]
    for _ in range(n - 1):
        r.step()
        want.append(r.tokens.clone())
    want = torch.stack(want, dim=1).tolist()
    model = models.load_model(str(tmp_path))
    engine = Engine(model, max_tokens=64 * 8, max_seqs=B)
    got = [o.tokens for o in engine.generate(prompts, SamplingParams(max_tokens=n))]
    assert got == want
    assert engine.cache.free_slots() == B and engine.cache.free_pages() == 8


def test_portions_and_mixed_batches(tmp_path):
    """Later portions run token by token over the 4-bit cache, so they agree with the whole prompt within its rounding."""
    _, cfg = ckpt.make_tiny_checkpoint(str(tmp_path), seed=4)
    tokens = np.random.default_rng(2).integers(0, cfg.vocab, 90).tolist()
    model = models.load_model(str(tmp_path))
    engine = Engine(model, max_tokens=64 * 8, max_seqs=3)

    def run(sizes):
        seq, at, out = engine.open(), 0, []
        for n in sizes:
            out.append(engine.run([SequenceInput(seq, tokens[at:at + n], list(range(n)))]))
            at += n
        engine.close(seq)
        return torch.cat(out)

    one = run([60] + [1] * 30)
    assert torch.allclose(run([60, 30]), one, atol=4e-3 * float(one.abs().max()))     # (the output head's product has other sizes)
    whole = run([90])
    assert (one - whole)[60:].norm() < 0.35 * whole[60:].norm() and torch.allclose(one[:60], whole[:60], atol=0.1 * float(one.abs().max()))
    a, b, c = engine.open(), engine.open(), engine.open()
    engine.run([SequenceInput(a, tokens[:60], [])])
    z = engine.run([SequenceInput(a, tokens[60:61], [0]), SequenceInput(b, tokens[:60], [59]), SequenceInput(c, tokens[:1], [0])])
    assert torch.allclose(z[:2], one[[60, 59]], atol=2e-2 * float(one.abs().max()))
    assert torch.allclose(z[2], one[0], atol=0.1 * float(one.abs().max()))


def test_command_line_generates(tmp_path, capsys):
    from omniserve_amd import cli
    _, cfg = ckpt.make_tiny_checkpoint(str(tmp_path), seed=5)
    assert cli.main(["generate", "--model", str(tmp_path), "--prompt-ids", "1,2,3", "--prompt-ids", "5", "--max-new-tokens", "4"]) == 0
    out = [json.loads(l) for l in capsys.readouterr().out.splitlines() if l.startswith("{")]
    assert [len(o["tokens"]) for o in out] == [4, 4] and out[0]["prompt"] == [1, 2, 3]
