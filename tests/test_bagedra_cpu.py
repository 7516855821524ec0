"""Bagedra without a GPU: configuration, batch tables of chunked and expanding layers, and the oracle by hand."""
import dataclasses
import json

import numpy as np
import pytest
import torch

from omniserve_amd import models
from omniserve_amd.engine.batch import BatchBuilder, Entry
from omniserve_amd.engine.cache import Cache
from omniserve_amd.models import bagedra, layers
from omniserve_amd.models.base import EngineModel
from oracle import bagedra as ref
from tests.bagedra_util import config, delta, gla, latent, random_state, tensors
from tests.hybrid_util import errors, to_numpy

CPU = torch.device("cpu")


def test_registry_and_config():
    assert models.model_class({"architecture": "Bagedra"}) is bagedra.Bagedra
    cfg = config([latent(base=777.0, scale=0.3), gla(tau=2.5), delta(conv=5, mlp=False), latent(kv_from=0, base=777.0, heads=2, dim=10, vdim=9, ff=33)],
                 width=72, vocab=33, eps=1e-3, embed_scale=7.0)
    spec = bagedra.parse_config(json.loads(json.dumps(cfg)))
    assert (spec.width, spec.vocab, spec.eps, spec.embed_scale, spec.norm, spec.placement) == (72, 33, 1e-3, 7.0, "rms", "after")
    a, b, c, d = (l.mixer for l in spec.layers)
    assert (a.kv_rank, a.rotary.dims, a.rotary.base, a.rotary.pairing, a.scale, a.kv_from) == (56, 12, 777.0, "halves", 0.3, None)
    assert (b.tau, c.taps, c.kv_heads, d.kv_from) == (2.5, 5, 2, 0)
    assert spec.layers[2].ff is None and spec.layers[3].ff == layers.DenseSpec(33, "gelu_tanh")


@pytest.mark.parametrize("bad", [
    [dict(latent(), type="other")], [dict(latent(), mlp={"kind": "moe"})], [latent(kv_from=0)], [gla(), latent(kv_from=0)],
    [latent(), latent(kv_from=1)], [latent(), latent(kv_from=0), latent(kv_from=1)], [latent(), latent(kv_from=0, kv_rank=8)],
    [latent(), latent(kv_from=0, base=5.0)], [latent(rot_dim=7)], [latent(scale=-1.0)], [delta(heads=3, kv_heads=2)], [delta(conv=0)],
    [gla(tau=0.0)], []], ids=str)
def test_configurations_that_make_no_sense(bad):
    with pytest.raises(ValueError):
        bagedra.parse_config(config(bad))


class Tables(EngineModel):
    vocab, dtype, device, chunk_rows, expand_pages = 9, torch.float32, CPU, 32, 4

    def kv_shapes(self):
        return [(1, 8, 0)]

    def state_shapes(self):
        return [(2, 4, 6), (3, 5)]


def test_batch_tables_of_chunks_and_expansions():
    m = Tables()
    cache, builder = Cache(m, 30, 6, CPU), BatchBuilder(m, CPU)
    assert cache.kv[0][0].shape == (30, 1, 64, 8) and cache.kv[0][1].numel() == 0
    assert [tuple(s.shape) for s in cache.state] == [(6, 2, 4, 6), (6, 3, 5)]
    seqs = [cache.open() for _ in range(5)]
    for s, n in zip(seqs, (0, 100, 63, 10, 300)):
        cache.reserve(s, n)
        cache.advance(s, n)
    counts = (33, 64, 2, 1, 40)
    for s, n in zip(seqs, counts):
        cache.reserve(s, n)
    b, _ = builder.build([Entry(s, [0] * n, []) for s, n in zip(seqs, counts)])
    assert b.n_entries == 4 and b.n_decode == 1
    ports, chunks = b.portions.tolist(), b.chunks.tolist()
    assert [p[:4] for p in ports] == [[0, 33, seqs[0].slot, 1], [33, 64, seqs[1].slot, 0], [97, 2, seqs[2].slot, 0], [99, 40, seqs[4].slot, 0]]
    assert [p[4:7] for p in ports] == [[0, 2, 0], [2, 2, 100], [4, 1, 63], [5, 2, 300]]
    assert chunks == [0, 0, 1, 1, 2, 3, 3]
    long = cache.open()
    cache.reserve(long, 700)
    s, _ = builder.build([Entry(seqs[3], [0, 0], []), Entry(long, [0] * 700, [])])
    assert s.multi_segment and s.segment_len == 256
    assert [x[:7] for x in s.segments.tolist()] == [[0, 2, seqs[3].slot, 0, 0, 1, 0]] + [
        [2 + 256 * i, n, long.slot, 1, i, 3, 1 + 8 * i] for i, n in enumerate((256, 256, 188))]
    # pages: 1, 3, 2, 6; at most 4 at once, one portion at least
    assert b.expansions == ((0, 4, 0, 2), (4, 2, 2, 1), (6, 6, 3, 1))
    pages, table = b.context_pages.tolist(), b.context_table.tolist()
    for k, (s, (page0, n, tile0, tiles)) in enumerate(zip((seqs[0], seqs[1], seqs[2], seqs[4]), [b.expansions[i] for i in (0, 0, 1, 2)])):
        assert [pages[page0 + i] for i in table[k][:s.pages]] == s.table[:s.pages].tolist()
        assert k in [e for e, _ in b.attn_tiles.tolist()[tile0:tile0 + tiles]]


def test_padding_of_single_sizes():
    assert [layers.pad_to(n, 64, 128, 192, 256) for n in (1, 64, 129, 192, 193)] == [64, 64, 192, 192, 256]
    with pytest.raises(ValueError):
        layers.pad_to(513, 64, 512)
    w = torch.randn((3 * 10, 7))
    p = layers.pad_out_heads(w, 3, 10, 8, 12)
    assert p.shape == (36, 8) and torch.equal(p.view(3, 12, 8)[:, :10, :7].reshape(30, 7), w) and not p.view(3, 12, 8)[:, 10:].any()


def test_oracle_recurrences_by_hand():
    one = np.ones((3, 1, 1))
    v = np.array([1.0, 2.0, 4.0]).reshape(3, 1, 1)
    o, s = ref.gated_linear_attention(one, one, v, np.log(np.array([0.5, 0.5, 0.25])).reshape(3, 1, 1))
    assert np.allclose(o.ravel(), [1.0, 2.5, 4.625]) and np.isclose(s[0, 0, 0], 4.625)
    # with a unit key the rule moves the state a step of beta towards v
    o, s = ref.gated_delta_rule(one, one, v, np.log(np.array([[1.0], [0.5], [1.0]])), np.array([[1.0], [0.5], [1.0]]))
    assert np.allclose(o.ravel(), [1.0, 0.5 + 0.5 * 1.5, 4.0])
    x = np.arange(1.0, 5.0)[:, None]
    assert ref.short_convolution(x, np.array([[100.0, 10.0, 1.0]]))[:, 0].tolist() == [1.0, 12.0, 123.0, 234.0]
    assert np.isclose(ref.gelu_tanh(1.0), 0.841192, atol=1e-6) and np.isclose(ref.softplus(0.0), np.log(2))
    turned = ref.rotate_halves(np.array([[[1.0, 2.0, 3.0, 4.0]]]), [1], np.array([np.pi / 2, 0.0]))
    assert np.allclose(turned, [[[-3.0, 2.0, 1.0, 4.0]]])


def test_oracle_latent_attention_by_hand():
    """Equal scores: the running mean of the values; one key far ahead of the others: its value."""
    q, c, kr = np.zeros((3, 1, 2)), np.array([[1.0], [3.0], [8.0]]), np.zeros((3, 1))
    o = ref.latent_attention(q, c, kr, np.ones((1, 1)), np.full((1, 1), 2.0), 1.0, 1, 1)
    assert np.allclose(o.ravel(), [2.0, 4.0, 8.0])
    q[2, 0, 1], kr[1, 0] = 10.0, 10.0
    o = ref.latent_attention(q, c, kr, np.ones((1, 1)), np.full((1, 1), 2.0), 1.0, 1, 1)
    assert np.isclose(o[2, 0, 0], 6.0)


def test_oracle_shares_latents_and_starts_from_the_residual():
    cfg = config([latent(), latent(kv_from=0)])
    w = to_numpy(random_state(cfg, 3))
    assert "l1.mix.dkv" not in w and set(w) == set(tensors(cfg))
    t = [5, 7, 11, 200]
    z, after = ref.decoder(cfg, w, t)
    alone = ref.decoder(dict(cfg, layers=cfg["layers"][:1]), w, t)[1]
    assert np.allclose(after[0], alone[0])
    w2 = dict(w, **{"l0.mix.dkv": 1.5 * w["l0.mix.dkv"][::-1]})
    assert errors(ref.decoder(cfg, w2, t)[0], z).min() > 1e-3


def test_specs_are_values():
    s = layers.LatentAttentionSpec(2, 8, 8, 16, layers.RotarySpec(4, 100.0, pairing="halves"), 0.5)
    assert dataclasses.replace(s, kv_from=0) != s
    with pytest.raises(ValueError):
        layers.AttentionSpec(2, 2, 8, 8, 1.0, rotary=layers.RotarySpec(4, 100.0, pairing="halves"))
