"""Lugasun without a GPU: configuration reading, registry, what goes over the ABI, and the oracle's mechanisms against brute force."""
import ctypes
import json
import math

import pytest
import torch

import lugasun_cases as LC
from callireader_amd import registry
from callireader_amd.config import DecoderSpec, DenseFF
from oracle import lugasun as O


def test_spec_reads_every_size_and_constant():
    s = DecoderSpec.from_lugasun(LC.RAGGED)
    assert (s.width, s.vocab, s.eps, s.loop, s.side_dim) == (184, 331, 1e-5, (1, 3, 3), 20)
    assert s.norm_plain and s.tied_head and s.loop_in and not s.post_norm and s.softcap == 0.0 and s.sinusoid_base == 0.0
    assert s.passes == [0, 1, 2, 1, 2, 1, 2] == [i for i, _ in O.passes(LC.RAGGED)]
    m = s.layers[1].mixer
    assert (m.left.heads, m.left.kv_heads, m.left.dim, m.left.vdim, m.left.chunk, m.left.scale, m.left.softcap, m.left.qk_norm) == (5, 1, 96, 112, 19, 0.2, 5.0, True)
    assert (m.left.rot.base, m.left.rot.dims, m.left_scale, m.right_scale) == (10000.0, 96, 1.3, 0.2)
    assert (m.right.heads, m.right.dim, m.right.vdim, m.right.decay, m.right.rot.base, m.right.rot.dims) == (2, 100, 33, (0.97, 0.995), 40.0, 36) and m.right.k_scale == 0.1
    assert s.layers[1].ff is None and s.layers[0].ff == DenseFF(200)
    shapes = s.weight_shapes()
    assert shapes['l0.mix.left.k'] == (120, 184) and shapes['l0.mix.left.v'] == (72, 184) and shapes['l2.mix.left.o'] == (184, 132) and shapes['l0.mix.left.q.norm'] == (40,)
    assert shapes['l1.mix.right.g'] == (66, 184) and shapes['l1.mix.right.o'] == (184, 66) and shapes['side.embed'] == (331, 60) and shapes['l2.side.proj'] == (184, 20)
    assert shapes['loop.in'] == (184, 368) and 'head' not in shapes and 'l1.norm2' not in shapes and 'l0.norm1b' not in shapes and shapes['l2.mlp.up'] == (72, 184)
    assert 'loop.in' not in DecoderSpec.from_lugasun(LC.WIDE).weight_shapes()
    assert DecoderSpec.from_lugasun(LC.TINY).layers[0].mixer.right.rot is None


def test_spec_refuses_what_it_does_not_know():
    for change, name in [(lambda c: c['layers'][0].update(type='serial'), 'serial'), (lambda c: c['layers'][0]['mlp'].update(kind='moe'), 'moe'),
                         (lambda c: c['layers'][0]['mixer']['right'].update(decay=[0.5] * 7), '7 decays')]:
        bad = json.loads(json.dumps(LC.TINY))
        change(bad)
        with pytest.raises(ValueError, match=name):
            DecoderSpec.from_lugasun(bad)


def test_registry_goes_by_config_json(tmp_path):
    (tmp_path / 'config.json').write_text(json.dumps(LC.TINY))
    assert registry.architecture(str(tmp_path)) == 'Lugasun' and registry.is_text_model(str(tmp_path))
    assert registry.model_class(str(tmp_path)).__name__ == 'LugasunForCausalLM'


def test_description_over_the_abi():
    """What DecoderEngine fills in for two mixers side by side; the decays outlive the call that made them."""
    import gc
    from callireader_amd import _binding as B
    from callireader_amd.engine import _describe_mixer
    s = DecoderSpec.from_lugasun(LC.RAGGED)
    layers = (B.LmLayer * 3)()
    for c, layer in zip(layers, s.layers):
        _describe_mixer(c, layer.mixer)
    gc.collect()
    c = layers[0]
    assert c.mixer == B.CR_MIX_HEADS | B.CR_MIX_RETENTION and c.attn.name == b'left.' and c.ret.name == b'right.'
    assert (c.attn.heads, c.attn.kv_heads, c.attn.dim, c.attn.vdim, c.attn.chunk, c.attn.qk_norm, c.attn.rot_dims, c.attn.rot_base) == (6, 3, 40, 24, 37, 1, 20, 3000.0)
    assert list(c.ret.decay[:3]) == [0.9, 1.0, 0.5] and list(layers[2].ret.decay[:5]) == [0.8] * 5
    assert abs(c.attn.out_scale - 0.7) < 1e-7 and abs(c.ret.out_scale - 0.4) < 1e-7 and abs(c.ret.k_scale - 24 ** -0.5) < 1e-7
    assert ctypes.sizeof(B.LmHeads) == 72 and ctypes.sizeof(B.LmRetention) == 56 and ctypes.sizeof(B.LmLayer) == 216 and ctypes.sizeof(B.LmDesc) == 92


def test_rotation_by_hand():
    x = torch.arange(1.0, 7.0).repeat(3, 1)[:, None, :]                # entries 0 .. 5, the first four turn: pairs (0, 2), (1, 3)
    y = O.rotate(x, 9.0, 4)
    assert torch.equal(y[0], x[0])
    for p in (1, 2):
        for i, f in ((0, 1.0), (1, 1.0 / 3.0)):
            c, s = math.cos(p * f), math.sin(p * f)
            u, v = i + 1.0, i + 3.0
            assert abs(float(y[p, 0, i]) - (u * c - v * s)) < 1e-5 and abs(float(y[p, 0, i + 2]) - (v * c + u * s)) < 1e-5
        assert y[p, 0, 4:].tolist() == [5.0, 6.0]
    assert torch.allclose(O.rotate(x[:1], 9.0, 4, start=2), y[2:])


def test_chunks_and_groups_by_brute_force():
    g = torch.Generator().manual_seed(0)
    n, H, G, d, dv = 11, 6, 2, 5, 3
    q, k, v = torch.randn(n, H, d, generator=g), torch.randn(n, G, d, generator=g), torch.randn(n, G, dv, generator=g)
    for size in (None, 1, 4, 11):
        o = O.grouped_attention(q, k, v, 0.7, 1.5, size)
        for i in range(n):
            for h in range(H):
                keys = [j for j in range(i + 1) if not size or i // size == j // size]
                s = [1.5 * math.tanh(0.7 * float(q[i, h] @ k[j, h // 3]) / 1.5) for j in keys]
                z = sum(math.exp(x) for x in s)
                want = sum(math.exp(x) / z * v[j, h // 3] for x, j in zip(s, keys))
                assert torch.allclose(o[i, h], want, atol=1e-5), (size, i, h)


def test_retention_is_the_decayed_sum():
    g = torch.Generator().manual_seed(1)
    q, k, v = torch.randn(9, 4, generator=g), torch.randn(9, 4, generator=g), torch.randn(9, 3, generator=g)
    for decay in (0.0, 0.5, 0.9, 1.0):
        o = O.decayed_recurrence(q, k, v, decay)
        for i in range(9):
            want = sum((decay ** (i - j) if i > j else 1.0) * float(q[i] @ k[j]) * v[j] for j in range(i + 1))
            assert torch.allclose(o[i], want, atol=1e-5)


def test_small_pieces_by_hand():
    assert torch.allclose(O.norm(torch.tensor([[3.0, 4.0]]), torch.tensor([1.0, 2.0]), 0.0), torch.tensor([[3.0, 8.0]]) / math.sqrt(12.5))
    w = {'m.up': torch.tensor([[1.0], [-1.0]]), 'm.down': torch.tensor([[1.0, 10.0]])}
    assert O.feed_forward(w, 'm.', torch.tensor([[3.0], [-2.0]])).flatten().tolist() == [9.0, 40.0]
    z = torch.linspace(-3, 3, 13)
    assert torch.allclose(O.gelu_tanh(z), torch.nn.functional.gelu(z, approximate='tanh'), atol=1e-6)
    x = torch.tensor([[1.0, 2.0]])
    w = {'side.embed': torch.tensor([[9.0, 9.0], [0.5, -3.0]]), 'l1.side.gate': torch.tensor([[1.0, 0.0]]), 'l1.side.proj': torch.tensor([[1.0], [2.0]]), 'l1.side.norm': torch.tensor([1.0, 0.5])}
    y = float(O.gelu_tanh(torch.tensor(1.0))) * -3.0                    # layer 1's single entry of token 1
    assert torch.allclose(O.token_side(w, 1, 1, x, torch.tensor([1]), 0.0), torch.tensor([[y, y]]) / math.sqrt((y * y + 4 * y * y) / 2))
    w = {'loop.in': torch.tensor([[1.0, 0.0, 0.0, 10.0], [0.0, 1.0, 0.0, 0.0]])}
    assert O.mix_in(w, torch.tensor([[1.0, 2.0]]), torch.tensor([[3.0, 4.0]])).tolist() == [[41.0, 2.0]]


def test_oracle_is_causal_and_loops_share_weights():
    cfg = LC.BIG
    w = LC.weights(cfg, 1)
    t = LC.tokens(cfg, 12)
    z, xs = O.forward(w, cfg, t, with_layers=True)
    assert len(xs) == 5 and O.passes(cfg) == [(0, True), (1, False), (0, True), (1, False), (2, False)]
    assert torch.allclose(z[:7], O.forward(w, cfg, t[:7]), atol=1e-4)
    assert not torch.allclose(O.forward(w, dict(cfg, loop=dict(start=0, stop=2, times=1)), t), z, atol=1e-2)


def test_bench_counts_work():
    from benchlib import decoder as D
    assert D._visible(10, 4) == 10 + 10 + 3 and D._visible(5, 0) == 15 and D._visible(5, 100) == 15
    s = DecoderSpec.from_lugasun(LC.TINY)
    W, per_layer = 64, 64 * 16 * 4 + 64 * 16 * 5 + 2 * 64 * 16 + 2 * 64 * 4      # attention, retention, feed-forward, token side
    weights = per_layer + 2 * W * W
    assert D.decode_bytes(s, 3, 9) == 2 * (weights + W * 40) + 2 * 3 * 2 * 32 + 8 * 3 * 256
    assert D.prefill_flops(s, 20, 2) == 2 * 20 * weights + 2 * 20 * 2 * 256 + 2 * 2 * D._visible(10, 8) * 32 + 2 * 2 * W * 40
