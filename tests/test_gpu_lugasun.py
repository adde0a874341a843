"""Lugasun on the GPU against the plain oracle (oracle/lugasun.py): float32 runs pin the mathematics, bfloat16 runs the served kernels.  float32 differences are rounding of sums
(bar 2e-5 of the logits' spread); bfloat16 bars are those of lugasun_cases.close, or stated where a test builds its own weights."""
import copy
import io
import json

import pytest
import torch

import lugasun_cases as LC
from oracle import lugasun as O

pytestmark = pytest.mark.gpu
F32, BF16 = torch.float32, torch.bfloat16
TOL = {F32: 2e-5, BF16: 4e-2}
CONFIGS = {'ragged': LC.RAGGED, 'wide': LC.WIDE, 'big': LC.BIG, 'huge': LC.HUGE, 'groups': LC.GROUPS, 'tiny': LC.TINY}


def model(cfg, w, dtype, max_tokens=1280, **kw):
    from callireader_amd.modeling_decoder import LugasunForCausalLM
    return LugasunForCausalLM.from_state_dict(w, cfg, dtype=dtype, max_tokens=max_tokens, **kw)


def logits_of(m, toks, portions=None, rid='r', keep=False):
    """All positions' logits, fed in `portions` (sizes; default: one prefill)."""
    out, at = [], 0
    for n in portions or [len(toks)]:
        out.append(m.step([(rid, toks[at:at + n], list(range(n)))]))
        at += n
    assert at == len(toks)
    if not keep:
        m.end(rid)
    return torch.cat(out).cpu()


def only(w, *keep):
    """Output projections at zero except those named: 'left', 'right', 'mlp', 'side'."""
    names = {'left.o': 'left', 'right.o': 'right', 'mlp.down': 'mlp', 'side.proj': 'side'}
    return {k: (torch.zeros_like(v) if any(k.endswith(n) and part not in keep for n, part in names.items()) else v) for k, v in w.items()}


# ---- whole prompts -------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize('dtype', [F32, BF16])
@pytest.mark.parametrize('name', CONFIGS)
def test_prompt(name, dtype):
    cfg = CONFIGS[name]
    w = LC.weights(cfg, 3, qk_gain=1.5 if dtype == F32 else 1.0)
    t = LC.tokens(cfg, 310 if name in ('wide', 'big') else 120)
    m = model(cfg, w, dtype)
    probe = m.engine.hidden_probe(len(t))
    z = logits_of(m, t)
    ref, xs = O.forward(w, cfg, t, with_layers=True)
    assert probe.shape[0] == len(xs) + 1
    for i, x in enumerate([w['embed'].float()[t]] + xs):
        assert LC.close(probe[i].cpu(), x, dtype), f'after pass {i}'
    assert LC.close(z, ref, dtype)
    m.close()


def test_large_prompts_take_the_tiled_kernels():
    """Enough rows for the persistent products, several 256-row retention chunks and 128-row blocks, in a batch of two: against the oracle and against a short prompt's kernels."""
    cfg = LC.config(256, 120, [LC.layer(LC.heads(4, 2, 64, 64, 700), LC.ret(64, 64, (0.999, 0.98)), 640), LC.layer(LC.heads(4, 2, 64, 64, 2000), LC.ret(128, 64, (0.9999,)), 512)], side=64, loop=(1, 2, 2))
    w = LC.weights(cfg, 26)
    m = model(cfg, w, BF16, max_tokens=1500, max_seqs=2)
    a, b = LC.tokens(cfg, 1410, 1), LC.tokens(cfg, 777, 2)
    z = m.step([('a', a, list(range(0, 1410, 7))), ('b', b, [0, 100, 776])]).cpu()
    m.end('a')
    m.end('b')
    za, zb = O.forward(w, cfg, a)[::7], O.forward(w, cfg, b)[[0, 100, 776]]
    assert LC.close(z, torch.cat([za, zb]), BF16)
    assert LC.close(logits_of(m, a[:90])[::7], za[:13], BF16)
    m.close()


# ---- mechanisms alone ----------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize('dtype', [F32, BF16])
@pytest.mark.parametrize('H,G,d,dv,size,cap,dims', [(3, 1, 40, 24, 64, 3.0, 40), (4, 4, 64, 64, 1, 9.0, 32), (16, 2, 128, 100, 130, 50.0, 128), (8, 1, 200, 256, 77, 2.0, 18), (2, 2, 300, 512, 40, 8.0, 2),
                                                   (33, 1, 20, 64, 5000, 0.7, 0)])
def test_attention_alone(H, G, d, dv, size, cap, dims, dtype):
    cfg = LC.config(192, 60, [LC.layer(LC.heads(H, G, d, dv, size, scale=1.3 / d ** 0.5, softcap=cap, rot=(300.0, dims)), LC.ret(16, 16, (0.9,)), None)], side=8)
    w = only(LC.weights(cfg, 6), 'left')
    t = LC.tokens(cfg, 200)
    m = model(cfg, w, dtype)
    probe = m.engine.hidden_probe(len(t))
    logits_of(m, t)
    x0, x1 = probe.cpu()
    added = cfg['layers'][0]['mixer']['left_scale'] * O.attention(w, 'l0.mix.left.', cfg['layers'][0]['mixer']['left'], O.norm(x0, w['l0.norm1'].float(), 1e-5), 1e-5)
    assert LC.rel(x1 - x0, added) < (1e-5 if dtype == F32 else 2e-2)
    m.close()


@pytest.mark.parametrize('dtype', [F32, BF16])
@pytest.mark.parametrize('d,dv,decay,dims', [(40, 24, (0.9, 0.99, 1.0), 40), (64, 64, (0.999,) * 5, 32), (128, 100, (0.5, 0.9999), 128), (200, 256, (0.97,), 18), (100, 130, (0.99,), 0),
                                            (300, 40, (0.98, 0.9), 300), (64, 400, (0.995,), 64)])
def test_retention_alone(d, dv, decay, dims, dtype):
    cfg = LC.config(192, 60, [LC.layer(LC.heads(1, 1, 16, 16, 8), LC.ret(d, dv, decay, rot=(300.0, dims)), None)], side=8)
    w = only(LC.weights(cfg, 7), 'right')
    t = LC.tokens(cfg, 600)
    m = model(cfg, w, dtype)
    probe = m.engine.hidden_probe(len(t))
    logits_of(m, t)
    x0, x1 = probe.cpu()
    added = cfg['layers'][0]['mixer']['right_scale'] * O.retention(w, 'l0.mix.right.', cfg['layers'][0]['mixer']['right'], O.norm(x0, w['l0.norm1'].float(), 1e-5), 1e-5)
    assert LC.rel(x1 - x0, added) < (2e-5 if dtype == F32 else 3e-2)
    m.close()


def test_extreme_decays_float32():
    """A decay of zero keeps the current token alone, a decay of one forgets nothing; neither is a special case."""
    cfg = LC.config(128, 60, [LC.layer(LC.heads(1, 1, 16, 16, 8), LC.ret(32, 32, (0.0, 1.0, 1e-30)), None)], side=8)
    w = only(LC.weights(cfg, 8), 'right')
    t = LC.tokens(cfg, 300)
    m = model(cfg, w, F32)
    ref = O.forward(w, cfg, t)
    assert LC.close(logits_of(m, t), ref, F32) and LC.close(logits_of(m, t, [150, 2, 100] + [1] * 48), ref, F32)
    m.close()


@pytest.mark.parametrize('dtype', [F32, BF16])
@pytest.mark.parametrize('ff', [16, 72, 512])
def test_feed_forward_alone(ff, dtype):
    cfg = LC.config(192, 60, [LC.layer(LC.heads(1, 1, 16, 16, 8), LC.ret(16, 16, (0.9,)), ff)], side=8)
    w = only(LC.weights(cfg, 9), 'mlp')
    t = LC.tokens(cfg, 90)
    m = model(cfg, w, dtype)
    probe = m.engine.hidden_probe(80)
    z = logits_of(m, t, [80] + [1] * 10)
    x0, x1 = probe.cpu()
    assert LC.rel(x1 - x0, O.feed_forward(w, 'l0.mlp.', O.norm(x0, w['l0.norm2'].float(), 1e-5))) < (1e-5 if dtype == F32 else 2e-2)
    assert LC.close(z, O.forward(w, cfg, t), dtype)
    m.close()


@pytest.mark.parametrize('dtype', [F32, BF16])
@pytest.mark.parametrize('side', [1, 24, 64, 200, 300])
def test_token_side_alone(side, dtype):
    """Three layers, each with its own part of the token's row; prompts and decoding."""
    cfg = LC.config(256, 60, [LC.layer(LC.heads(1, 1, 16, 16, 8), LC.ret(16, 16, (0.9,)), 16 if i else None) for i in range(3)], side=side, loop=(1, 3, 2))
    w = only(LC.weights(cfg, 10), 'side')
    t = LC.tokens(cfg, 80)
    ref, xs = O.forward(w, cfg, t, with_layers=True)
    m = model(cfg, w, dtype)
    probe = m.engine.hidden_probe(70)
    z = logits_of(m, t, [70] + [1] * 10)
    for i, x in enumerate(xs):
        assert LC.rel(probe[i + 1].cpu(), x[:70]) < (1e-5 if dtype == F32 else 6e-2), i
    assert LC.close(z, ref, dtype)
    m.close()


@pytest.mark.parametrize('dtype', [F32, BF16])
@pytest.mark.parametrize('loop', [(0, 1, 1), (0, 2, 3), (1, 2, 2), (2, 3, 4), None])
def test_loop_entry(loop, dtype):
    """Where the span starts and how often it runs; no span means no entry product.  Nothing but the entries and the token side changes the stream."""
    cfg = LC.config(136, 60, [LC.layer(LC.heads(1, 1, 16, 16, 8), LC.ret(16, 16, (0.9,)), None) for _ in range(3)], side=8, loop=loop)
    w = only(LC.weights(cfg, 11), 'side')
    t = LC.tokens(cfg, 30)
    ref, xs = O.forward(w, cfg, t, with_layers=True)
    m = model(cfg, w, dtype)
    probe = m.engine.hidden_probe(20)
    z = logits_of(m, t, [20] + [1] * 10)
    assert probe.shape[0] == len(xs) + 1
    for i, x in enumerate(xs):
        assert LC.rel(probe[i + 1].cpu(), x[:20]) < (1e-5 if dtype == F32 else 6e-2), i
    assert LC.close(z, ref, dtype)
    m.close()


def test_squared_relu_products():
    """The epilogue in every kernel that has it: 128- and 256-row tiles, the tail rows' kernel, the weight-streaming kernels."""
    from callireader_amd.engine import op_gemm
    g = torch.Generator().manual_seed(0)
    for M, N, K in [(3, 96, 128), (40, 200, 256), (33, 8256, 2048), (64, 16384, 256), (300, 72, 64), (2048 + 40, 1024, 256), (4096, 520, 128)]:
        A, W = torch.randn(M, K, generator=g).to(BF16), (torch.randn(N, K, generator=g) / K ** 0.5).to(BF16)
        C = op_gemm(12, A.cuda(), W.cuda()).float().cpu()
        ref = torch.relu(A.float() @ W.float().T).square()
        assert float((C - ref).abs().max()) < 2 ** -8 * float(ref.max()), (M, N, K)


def test_positions_far_out_float32():
    """Rotations at positions in the thousands, in attention and in retention."""
    cfg = LC.config(96, 64, [LC.layer(LC.heads(2, 1, 32, 16, 4096, rot=(20000.0, 32)), LC.ret(32, 16, (0.9995,), rot=(1e6, 32)), None)], side=4)
    w = LC.weights(cfg, 12)
    t = LC.tokens(cfg, 4200)
    m = model(cfg, w, F32, max_tokens=4224)
    z = m.step([('r', t[:4190], list(range(4000, 4190)))]).cpu()
    z = torch.cat([z] + [m.step([('r', [x], [0])]).cpu() for x in t[4190:]])
    assert LC.rel(z, O.forward(w, cfg, t)[4000:]) < 2e-4          # an angle of 4000 radians has 2e-4 radians of fp32 rounding
    m.close()


# ---- the cache and the state ---------------------------------------------------------------------------------------------------
@pytest.mark.parametrize('dtype', [F32, BF16])
@pytest.mark.parametrize('name', ['ragged', 'wide', 'big', 'huge', 'groups'])
def test_decoding_equals_the_prompt(name, dtype):
    """Token by token from the first token on, against the prompt in one piece."""
    cfg = CONFIGS[name]
    w = LC.weights(cfg, 11, qk_gain=1.5 if dtype == F32 else 1.0)
    t = LC.tokens(cfg, 100)
    m = model(cfg, w, dtype)
    one = logits_of(m, t)
    by_one = logits_of(m, t, [1] * 100)
    ref = O.forward(w, cfg, t)
    assert LC.close(by_one, ref, dtype) and LC.close(by_one, one, dtype)
    m.close()


@pytest.mark.parametrize('dtype', [F32, BF16])
@pytest.mark.parametrize('sizes', [[2] * 20, [1, 2, 37], [7, 7, 7, 7, 7, 5], [39, 1], [3, 1, 1, 30, 2, 3]])
@pytest.mark.parametrize('name', ['ragged', 'big'])
def test_portions(name, sizes, dtype):
    cfg = CONFIGS[name]
    w = LC.weights(cfg, 12)
    t = LC.tokens(cfg, 40)
    m = model(cfg, w, dtype)
    assert LC.close(logits_of(m, t, sizes), O.forward(w, cfg, t), dtype)
    m.close()


@pytest.mark.parametrize('dtype', [F32, BF16])
@pytest.mark.parametrize('sizes', [[255, 2, 255, 8], [256, 256, 8], [257, 263], [64, 64, 2, 390], [1, 519], [500, 20]])
def test_long_portions(sizes, dtype):
    """Portions that end before, at and behind the edges of attention chunks (150, 300), retention chunks (256 rows) and tiles (64)."""
    cfg = LC.WIDE
    w = LC.weights(cfg, 13)
    t = LC.tokens(cfg, 520)
    m = model(cfg, w, dtype)
    assert LC.close(logits_of(m, t, sizes), O.forward(w, cfg, t), dtype)
    m.close()


@pytest.mark.parametrize('dtype', [F32, BF16])
def test_batch_of_unequal_requests(dtype):
    """Each request in a batch gets what it gets alone: prompts of 1 to 330 tokens, decoded together, the short ones leaving early; then portions in a mixed batch."""
    cfg = LC.WIDE
    w = LC.weights(cfg, 13)
    m = model(cfg, w, dtype, max_seqs=5)
    lens = [1, 330, 17, 149, 65]
    toks = [LC.tokens(cfg, n + 12, seed=n) for n in lens]
    alone = [logits_of(m, t) for t in toks]
    got = [[] for _ in lens]
    z = m.step([(i, t[:n], [n - 1]) for i, (t, n) in enumerate(zip(toks, lens))]).cpu()
    for i in range(5):
        got[i].append(z[i])
    live = list(range(5))
    for k in range(12):
        z = m.step([(i, [toks[i][lens[i] + k]], [0]) for i in live]).cpu()
        for j, i in enumerate(live):
            got[i].append(z[j])
        if k in (3, 7):
            m.end(live.pop(0))
    for i, n in enumerate(lens):
        g = torch.stack(got[i])
        assert LC.close(g, alone[i][n - 1:n - 1 + len(g)], dtype), i
    for i in live:
        m.end(i)
    m.step([('p', toks[1][:50], []), ('q', toks[3][:9], [])])                    # two caches of different length, then portions of different length in one step
    z = m.step([('q', toks[3][9:60], [50]), ('p', toks[1][50:52], [1])]).cpu()
    assert LC.close(z[0:1], alone[3][59:60], dtype) and LC.close(z[1:2], alone[1][51:52], dtype)
    z = m.step([('p', toks[1][52:200], [147]), ('q', toks[3][60:151], [90])]).cpu()      # both portions cross a chunk's edge
    assert LC.close(z[0:1], alone[1][199:200], dtype) and LC.close(z[1:2], alone[3][150:151], dtype)
    m.close()


@pytest.mark.parametrize('dtype', [F32, BF16])
@pytest.mark.parametrize('name', ['ragged', 'big'])
def test_slots_used_again(name, dtype):
    """A slot that held a longer request gives a shorter one nothing of it -- no key, no state -- in prompts and in decoding from the first token on."""
    cfg = CONFIGS[name]
    w = LC.weights(cfg, 14)
    m = model(cfg, w, dtype, max_seqs=2)
    long_, short = LC.tokens(cfg, 200, 1), LC.tokens(cfg, 30, 2)
    ref = O.forward(w, cfg, short)
    for sizes in ([20] + [1] * 10, [1] * 30):
        m.step([('long', long_, []), ('other', long_[:90], [])])
        m.end('long')
        m.end('other')
        assert LC.close(logits_of(m, short, sizes), ref, dtype)
    m.step([('long', long_, []), ('other', long_[:90], [])])
    m.end('long')                                                                # one slot free, the other in use
    assert LC.close(logits_of(m, short, [20] + [1] * 10), ref, dtype)
    m.close()


@pytest.mark.parametrize('dtype', [F32, BF16])
def test_first_tokens(dtype):
    cfg = LC.RAGGED
    w = LC.weights(cfg, 15)
    m = model(cfg, w, dtype)
    for n in (1, 2, 3):
        t = LC.tokens(cfg, n, seed=n)
        ref = O.forward(w, cfg, t)
        assert LC.close(logits_of(m, t), ref, dtype)
        assert LC.close(logits_of(m, t, [1] * n), ref, dtype)
    m.close()


PLANTED = 0


def planted_key(size, dim=48, H=4, G=2):
    """One attention layer whose queries all look for ONE planted token (used nowhere else): a weight close to one on its key wherever it is visible, so a lost, shifted or doubled
    key shows at once and rounding does not.  Entry 100 of every embedding is alike (queries look at it), entry 101 marks the planted token."""
    cfg = LC.config(128, 50, [LC.layer(LC.heads(H, G, dim, 40, size, scale=1.0, softcap=45.0, rot=(10.0, 16)), LC.ret(16, 16, (0.9,)), None, (1.0, 1.0))], side=4)
    w = only(LC.weights(cfg, 16), 'left')
    e = w['embed'].float()
    e[:, 100], e[:, 101], e[PLANTED, 101] = 4.0, 0.0, 12.0
    q, k = 0.05 * w['l0.mix.left.q'].float(), 0.05 * w['l0.mix.left.k'].float()
    k[:, 101] = 0.0
    q[dim - 1::dim, :], k[dim - 1::dim, :] = 0.0, 0.0
    q[dim - 1::dim, 100], k[dim - 1::dim, 101] = 2.0, 2.0             # an entry of the head that no rotation touches
    w.update({'embed': e.to(BF16), 'l0.norm1': torch.ones(128, dtype=BF16), 'l0.mix.left.q': q.to(BF16), 'l0.mix.left.k': k.to(BF16), 'l0.mix.left.q.norm': torch.ones(dim, dtype=BF16),
              'l0.mix.left.k.norm': torch.ones(dim, dtype=BF16), 'final.norm': torch.full((128,), 0.1, dtype=BF16)})
    return cfg, w


def others(cfg, n, seed):
    return [t if t != PLANTED else 1 for t in LC.tokens(cfg, n, seed)]


@pytest.mark.parametrize('dtype', [F32, BF16])
@pytest.mark.parametrize('size', [100, 64, 333])
def test_a_planted_key_is_seen_in_its_chunk_and_nowhere_else(size, dtype):
    """Just inside and just outside every chunk edge, from prompts in one piece, from a portion that starts inside the chunk, and from decoding across the edge."""
    n = 2 * size + 60
    cfg, w = planted_key(size)
    m = model(cfg, w, dtype, max_tokens=n)
    base = others(cfg, n, 18)
    plain = O.forward(w, cfg, base)
    for at in (0, 1, size - 1, size, size + 1, 2 * size - 1, 2 * size):
        t = list(base)
        t[at] = PLANTED
        ref = O.forward(w, cfg, t)
        shows = (ref - plain).pow(2).mean(-1).sqrt() / plain.std()
        end = (at // size + 1) * size
        assert float(shows[at + 1:end].min() if end > at + 1 else 1.0) > 0.3, 'the planted key does not show'
        assert end >= n or float(shows[end:].max()) == 0.0
        cut = end - 5 if end <= n else n - 20
        for sizes in ([n], [max(at - 3, 1), n - max(at - 3, 1)], [cut] + [1] * 30 + [n - cut - 30] if n - cut > 30 else [cut] + [1] * (n - cut)):
            assert LC.rel(logits_of(m, t, sizes), ref) < TOL[dtype], (at, sizes)
    m.close()


@pytest.mark.parametrize('dtype', [F32, BF16])
def test_a_planted_key_far_away(dtype):
    """One chunk of many tiles (64 keys), blocks (128 rows) and decode splits (256 keys): the key at their edges, seen from far behind, in prompts and in decoding."""
    n = 1030
    cfg, w = planted_key(5000)
    m = model(cfg, w, dtype, max_tokens=1100)
    base = others(cfg, n + 6, 18)
    plain = O.forward(w, cfg, base)
    for at in (0, 1, 31, 32, 63, 64, 127, 128, 255, 256, 511, 512, 513, 1022, 1023, 1024):
        t = list(base)
        t[at] = PLANTED
        ref = O.forward(w, cfg, t)
        a = m.step([('r', t[:n], list(range(n - 4, n)))]).cpu()
        b = torch.cat([m.step([('r', [t[n + k]], [0])]) for k in range(6)]).cpu()
        m.end('r')
        z, want = torch.cat([a, b]), ref[n - 4:n + 6]
        shows = (want - plain[n - 4:n + 6]).pow(2).mean(-1).sqrt() / plain.std()
        assert float(shows[max(0, at - n + 5):].min()) > 0.3, 'the planted key does not show'
        assert LC.rel(z, want) < TOL[dtype], at
    m.close()


def planted_memory(decay, dim=48, vdim=40):
    """One retention layer in which only the planted token writes (every other key is nearly nothing) and every query reads it: what is read decays but its direction, which the
    norm over the head leaves, is the planted value's."""
    cfg = LC.config(128, 50, [LC.layer(LC.heads(1, 1, 16, 16, 8), LC.ret(dim, vdim, decay, rot=(10.0, 16)), None, (1.0, 1.0))], side=4, eps=1e-12)
    w = only(LC.weights(cfg, 17), 'right')
    e = w['embed'].float()
    e[:, 100], e[:, 101], e[PLANTED, 101] = 4.0, 0.0, 12.0
    q, k = 0.05 * w['l0.mix.right.q'].float(), 0.0 * w['l0.mix.right.k'].float()
    q[dim - 1::dim, 100], k[dim - 1::dim, 101], k[dim - 1::dim, 100] = 2.0, 2.0, 1e-6
    w.update({'embed': e.to(BF16), 'l0.norm1': torch.ones(128, dtype=BF16), 'l0.mix.right.q': q.to(BF16), 'l0.mix.right.k': k.to(BF16), 'final.norm': torch.full((128,), 0.1, dtype=BF16)})
    return cfg, w


@pytest.mark.parametrize('dtype', [F32, BF16])
@pytest.mark.parametrize('dims', [(48, 40), (128, 128), (256, 200), (60, 300)])
def test_a_planted_memory_is_kept(dims, dtype):
    """Written at the edges of tiles, blocks and 256-row chunks, read hundreds of tokens on: in one piece, over portions, and in decoding."""
    n = 700
    cfg, w = planted_memory((0.99, 1.0, 0.997), *dims)
    m = model(cfg, w, dtype, max_tokens=n)
    base = others(cfg, n, 19)
    plain = O.forward(w, cfg, base)
    for at in (0, 1, 63, 64, 255, 256, 257, 511, 512):
        t = list(base)
        t[at] = PLANTED
        ref = O.forward(w, cfg, t)
        shows = (ref - plain).pow(2).mean(-1).sqrt() / plain.std()
        assert float(shows[at + 1:].min()) > 0.2, 'the planted token does not show'
        for sizes in ([n], [max(at - 1, 1), 2, n - 2 - max(at - 1, 1)], [at + 1, 40] + [1] * 20 + [n - at - 61]):
            assert LC.rel(logits_of(m, t, sizes), ref) < TOL[dtype], (at, sizes)
    m.close()


@pytest.mark.parametrize('dtype', [F32, BF16])
def test_decoding_across_edges_together(dtype):
    """Two sequences at different lengths decode in the same steps, one over a chunk's edge (300), one over a 256-key split's."""
    cfg = LC.config(192, 90, [LC.layer(LC.heads(8, 2, 64, 64, 300), LC.ret(64, 32, (0.99, 0.95)), 64), LC.layer(LC.heads(6, 1, 32, 40, 1000), LC.ret(32, 64, (0.999,)), None)], side=16)
    w = LC.weights(cfg, 19)
    t, s = LC.tokens(cfg, 305, 1), LC.tokens(cfg, 262, 2)
    m = model(cfg, w, dtype, max_seqs=2)
    m.step([('a', t[:295], []), ('b', s[:252], [])])
    za, zb = [], []
    for k in range(10):
        z = m.step([('a', [t[295 + k]], [0]), ('b', [s[252 + k]], [0])]).cpu()
        za.append(z[0])
        zb.append(z[1])
    assert LC.close(torch.stack(za), O.forward(w, cfg, t)[295:], dtype)
    assert LC.close(torch.stack(zb), O.forward(w, cfg, s)[252:], dtype)
    m.close()


@pytest.mark.parametrize('dtype', [F32, BF16])
def test_long_decoding(dtype):
    cfg = LC.TINY
    w = LC.weights(cfg, 20)
    t = LC.tokens(cfg, 400)
    m = model(cfg, w, dtype)
    assert LC.close(logits_of(m, t, [1] * 400), O.forward(w, cfg, t), dtype)
    m.close()


def test_long_state_decoding():
    """A state that forgets nothing over a thousand decoded tokens: the carried sum is fp32 in both types."""
    cfg = LC.config(128, 60, [LC.layer(LC.heads(1, 1, 16, 16, 8), LC.ret(64, 64, (1.0, 0.9999)), None)], side=4)
    w = only(LC.weights(cfg, 21), 'right')
    t = LC.tokens(cfg, 1040)
    ref = O.forward(w, cfg, t)
    for dtype in (F32, BF16):
        m = model(cfg, w, dtype)
        m.step([('r', t[:20], [])])
        z = torch.cat([m.step([('r', [x], [0])]) for x in t[20:]]).cpu()
        assert LC.close(z, ref[20:], dtype)
        m.close()


def test_more_decode_rows_than_the_streaming_kernels_take():
    """70 sequences decode together (tiled kernels) and 5 of them alone (weight-streaming kernels): the same logits beyond rounding."""
    cfg = LC.WIDE
    w = LC.weights(cfg, 21)
    m = model(cfg, w, BF16, max_tokens=64, max_seqs=70)
    toks = [LC.tokens(cfg, 4 + i % 9, seed=i) for i in range(70)]
    m.step([(i, t[:-1], []) for i, t in enumerate(toks)])
    z = m.step([(i, t[-1:], [0]) for i, t in enumerate(toks)]).cpu()
    for i in range(70):
        m.end(i)
    for i in (0, 8, 33, 64, 69):
        assert LC.close(z[i:i + 1], O.forward(w, cfg, toks[i])[-1:], BF16)
        assert LC.close(z[i:i + 1], logits_of(m, toks[i], [len(toks[i]) - 1, 1])[-1:], BF16)
    m.close()


def test_decode_batches_of_every_kernel_form():
    """1, 9, 17, 40 and 64 rows of a width whose fused projection and feed-forward take the N-split streaming kernel: every row as alone."""
    cfg = LC.config(2048, 200, [LC.layer(LC.heads(16, 4, 128, 128, 100), LC.ret(128, 128, (0.97,) * 11), 8320)], side=128, loop=(0, 1, 1))
    w = LC.weights(cfg, 22)
    m = model(cfg, w, BF16, max_tokens=64, max_seqs=64)
    toks = [LC.tokens(cfg, 3 + i % 5, seed=i) for i in range(64)]
    ref = torch.cat([O.forward(w, cfg, t)[-1:] for t in toks])
    for rows in (1, 9, 17, 40, 64):
        m.step([(i, toks[i][:-1], []) for i in range(rows)])
        z = m.step([(i, toks[i][-1:], [0]) for i in range(rows)]).cpu()
        for i in range(rows):
            m.end(i)
        assert LC.close(z, ref[:rows], BF16), rows
    m.close()


# ---- a mixer of either kind on its own, through the same description -------------------------------------------------------------
@pytest.mark.parametrize('dtype', [F32, BF16])
@pytest.mark.parametrize('kind', ['attention', 'retention'])
def test_one_mixer_in_a_layer(kind, dtype):
    """The description's parts are independent: attention over heads without chunks, cap, query norms or rotation, or retention alone; untied head, no token side, no loop."""
    from callireader_amd.config import DecoderLayer, DecoderSpec, DenseFF, HeadsMixer, RetentionMixer
    mixer = HeadsMixer(heads=6, kv_heads=2, dim=32, vdim=48, scale=0.2) if kind == 'attention' else RetentionMixer(heads=3, dim=32, vdim=48, decay=(0.9, 0.95, 0.99), k_scale=0.1)
    spec = DecoderSpec(width=128, vocab=90, layers=(DecoderLayer(mixer, DenseFF(192)),), eps=1e-5, norm_plain=True, post_norm=False)
    g = torch.Generator().manual_seed(0)
    w = {k: ((1 + 0.2 * torch.randn(s, generator=g)) if len(s) == 1 else torch.randn(s, generator=g) / (1 if k == 'embed' else s[1] ** 0.5)).to(BF16) for k, s in spec.weight_shapes().items()}
    assert 'head' in w and 'l0.mix.q' in w and 'side.embed' not in w
    t = torch.randint(0, 90, (300,), generator=g).tolist()
    x = w['embed'].float()[t]
    h = O.norm(x, w['l0.norm1'].float(), 1e-5)
    if kind == 'attention':
        q, k, v = ((h @ w['l0.mix.' + n].float().T).view(300, c, d) for n, c, d in (('q', 6, 32), ('k', 2, 32), ('v', 2, 48)))
        x = x + O.grouped_attention(q, k, v, 0.2, None, None).reshape(300, -1) @ w['l0.mix.o'].float().T
    else:
        q, k, v = ((h @ w['l0.mix.' + n].float().T).view(300, 3, d) for n, d in (('q', 32), ('k', 32), ('v', 48)))
        gate = h @ w['l0.mix.g'].float().T
        o = torch.stack([O.rms(O.decayed_recurrence(q[:, i], 0.1 * k[:, i], v[:, i], mixer.decay[i]), 1e-5) for i in range(3)], 1)
        x = x + (o.reshape(300, -1) * gate * torch.sigmoid(gate)) @ w['l0.mix.o'].float().T
    x = x + O.feed_forward(w, 'l0.mlp.', O.norm(x, w['l0.norm2'].float(), 1e-5))
    ref = O.norm(x, w['final.norm'].float(), 1e-5) @ w['head'].float().T
    m = model(spec, w, dtype)
    assert LC.close(logits_of(m, t), ref, dtype) and LC.close(logits_of(m, t, [260, 2] + [1] * 38), ref, dtype)
    m.close()


# ---- generation ----------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize('dtype', [F32, BF16])
def test_generate_is_the_greedy_continuation(dtype):
    """The framework's own entry point and scheduler: a batch of unequal prompts, EOS inside, one id at a time otherwise.  bf16: up to the first pick the oracle itself calls close."""
    cfg = LC.BIG
    w = LC.weights(cfg, 28, out_gain=3.0)
    prompts = [LC.tokens(cfg, n, seed=30 + n) for n in (5, 1, 60, 9, 23)]
    m = model(cfg, w, dtype)
    got = m.generate(prompts, max_new_tokens=20, check_every=3)
    ref = [O.greedy(w, cfg, p, 20) for p in prompts]
    sures = 0
    for g, (ids, margins) in zip(got, ref):
        assert len(g) == 20
        bar = 1e-4 if dtype == F32 else 0.2
        sure = next((i for i, x in enumerate(margins) if x < bar), 20)
        assert g[:sure] == ids[:sure], (sure, g, ids)
        sures += sure
    assert sures >= (100 if dtype == F32 else 12)
    if dtype == F32:
        eos = ref[0][0][7]
        stop = [O.greedy(w, cfg, p, 20, eos) for p in prompts]
        assert m.generate(prompts, max_new_tokens=20, eos_token_id=eos, check_every=4) == [ids for ids, _ in stop]
        assert m.generate([prompts[2]], max_new_tokens=20) == [ref[2][0]]            # alone, on a slot used before
    with pytest.raises(ValueError):
        m.generate([[1] * 5], max_new_tokens=5000)
    m.close()


def saved(tmp_path, cfg, w):
    from safetensors.torch import save_file
    (tmp_path / 'config.json').write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / 'model.safetensors'))
    return str(tmp_path)


def test_checkpoint_directory_to_ids(tmp_path):
    """config.json + model.safetensors -> registry -> weights -> generate, and the command line on the same directory."""
    from callireader_amd import inference, registry
    cfg = LC.RAGGED
    w = LC.weights(cfg, 24, out_gain=2.0)
    path = saved(tmp_path, cfg, w)
    m = registry.model_class(path).from_pretrained(path, dtype=F32, max_tokens=128)
    p = [3, 200, 17, 5]
    got = m.generate([p], max_new_tokens=8)
    m.close()
    ids, margins = O.greedy(w, cfg, p, 8)
    assert min(margins) > 1e-3 and got == [ids]
    out = inference.main(['--model', path, '--prompt_ids', '3,200,17,5', '--prompt_ids', '9', '--max_new_tokens', '8', '--dtype', 'float32'])
    assert out[0] == ids and len(out[1]) == 8


def test_a_replayed_trace(tmp_path):
    """The trace runner: steps in, logits files and `done` lines out."""
    import numpy as np
    from callireader_amd import trace
    cfg = LC.RAGGED
    w = LC.weights(cfg, 25)
    path = saved(tmp_path, cfg, w)
    a, b = LC.tokens(cfg, 42, 1), LC.tokens(cfg, 6, 2)
    steps = [dict(step=0, entries=[dict(id='a', tokens=a[:40], want=[0, 39]), dict(id='b', tokens=b[:4], want=[])], end=[]),
             dict(step=1, entries=[dict(id='a', tokens=a[40:41], want=[]), dict(id='b', tokens=b[4:5], want=[0])], end=['b']),
             dict(step=2, entries=[dict(id='a', tokens=a[41:], want=[0])], end=['a']),
             dict(step=3, entries=[dict(id='b', tokens=b, want=[5]), dict(id='c', tokens=a[:3], want=[2]), dict(id='d', tokens=a[:1], want=[])], end=[])]
    out = io.StringIO()
    assert trace.main(['--model', path, '--dtype', 'float32', '--out', path, '--max-tokens', '64'], stdin=io.StringIO('\n'.join(map(json.dumps, steps)) + '\n'), stdout=out) == 0
    assert out.getvalue().split('\n')[:4] == [f'done {i}' for i in range(4)]
    za, zb = O.forward(w, cfg, a), O.forward(w, cfg, b)
    want = [torch.stack([za[0], za[39]]), zb[4:5], za[41:42], torch.stack([zb[5], za[2]])]
    for i, ref in enumerate(want):
        z = torch.from_numpy(np.fromfile(tmp_path / f'{i}.f32', '<f4').reshape(len(ref), -1))
        assert LC.close(z, ref, F32), i


def test_a_second_context_borrows_the_weights():
    """cr_share_weights: another context decodes on the first one's weights, cache and states, until the owner's weights change."""
    from callireader_amd._binding import CalliReaderError
    from callireader_amd.engine import DecoderEngine
    cfg = LC.BIG
    w = LC.weights(cfg, 27)
    t = LC.tokens(cfg, 40)
    m = model(cfg, w, F32)
    m.step([('r', t[:39], [])])
    e2 = DecoderEngine(m.spec, dtype=F32)
    e2.share_weights_from(m.engine)
    z = e2.decode(m.slots.kv, [m.slots.slot['r']], force_tokens=torch.tensor([t[39]]), want_logits=True)
    assert LC.close(z.cpu(), O.forward(w, cfg, t)[-1:], F32)
    m.engine.load_state_dict(w)
    m.engine.finalize()
    with pytest.raises(CalliReaderError, match='share again'):
        e2.decode(m.slots.kv, [0], force_tokens=torch.tensor([1]))
    z = m.engine.decode(m.slots.kv, [m.slots.slot['r']], force_tokens=torch.tensor([3]), want_logits=True).cpu()
    assert LC.close(z, O.forward(w, cfg, t + [3])[-1:], F32)                 # the owner goes on, on the reloaded weights
    e2.close()
    m.close()


def test_errors_come_from_the_host():
    from callireader_amd._binding import CalliReaderError
    cfg = LC.TINY
    m = model(cfg, LC.weights(cfg), F32, max_tokens=16)
    with pytest.raises(CalliReaderError, match='vocabulary'):
        m.step([('a', [cfg['vocab']], [])])
    with pytest.raises(CalliReaderError, match='exceed the cache'):
        m.step([('a', [1] * 17, [])])
    m.close()
    w = LC.weights(cfg)
    del w['l0.mix.right.g']
    with pytest.raises(KeyError, match='l0.mix.right.g'):
        model(cfg, w, F32)
    for change in (dict(dim=600), dict(kv_heads=3), dict(rot=dict(base=10.0, dims=3)), dict(rot=dict(base=10.0, dims=40))):
        bad = copy.deepcopy(LC.TINY)
        bad['layers'][0]['mixer']['left'].update(change)
        with pytest.raises(CalliReaderError, match='layer 0'):
            model(bad, {}, F32)
