"""Small Lugasun configurations and seeded weights of the tests' own (several sizes that no kernel tile divides, layers that differ from each other)."""
import math

import torch


def heads(H, G, dim, vdim, size, scale=None, softcap=12.0, rot=(10000.0, None)):
    return dict(heads=H, kv_heads=G, dim=dim, vdim=vdim, mask=dict(size=size), scale=dim ** -0.5 if scale is None else scale, softcap=softcap,
                rot=dict(base=rot[0], dims=dim if rot[1] is None else rot[1]))


def ret(dim, vdim, decay, rot=(500.0, None)):
    return dict(heads=len(decay), dim=dim, vdim=vdim, decay=list(decay), rot=dict(base=rot[0], dims=dim if rot[1] is None else rot[1]))


def layer(left, right, ff, scales=(0.7, 0.4)):
    return dict(type='parallel', mixer=dict(left=left, right=right, left_scale=scales[0], right_scale=scales[1]), mlp=dict(kind='dense', ff=ff) if ff else None)


def config(width, vocab, layers, side, loop=None, eps=1e-5):
    return dict(architecture='Lugasun', width=width, vocab=vocab, norm=dict(eps=eps), layers=layers, token_side=dict(dim=side),
                **({'loop': dict(start=loop[0], stop=loop[1], times=loop[2])} if loop else {}))


# layers of three shapes (one without a feed-forward, rotations of a part of the head and of odd halves, a decay of one), the span 1 .. 2 looped three times
RAGGED = config(184, 331, [layer(heads(6, 3, 40, 24, 37, rot=(3000.0, 20)), ret(24, 52, (0.9, 1.0, 0.5)), 200),
                           layer(heads(5, 1, 96, 112, 19, scale=0.2, softcap=5.0), ret(100, 33, (0.97, 0.995), rot=(40.0, 36)), None, (1.3, 0.2)),
                           layer(heads(4, 4, 24, 33, 70, rot=(77.0, 6)), ret(16, 16, (0.8,) * 5), 72)], side=20, loop=(1, 3, 3))
# matrix-core instances: 128-wide heads in groups of four, 128 x 128 states
WIDE = config(256, 260, [layer(heads(8, 2, 128, 128, 150), ret(128, 128, (0.99, 0.9995, 0.93)), 320), layer(heads(8, 2, 128, 96, 300, softcap=30.0), ret(90, 128, (0.98, 0.6)), 64)], side=64)
# 256-wide heads and states, more value than key columns and the other way round
BIG = config(192, 130, [layer(heads(2, 1, 200, 232, 90), ret(250, 200, (0.99, 0.9)), 96), layer(heads(3, 3, 256, 130, 64), ret(40, 256, (0.95,)), 192),
                        layer(heads(2, 2, 64, 64, 45), ret(192, 40, (0.97, 0.992)), 128)], side=24, loop=(0, 2, 2))
# past the matrix-core instances: attention heads of 300, states of 300 x 400
HUGE = config(128, 90, [layer(heads(2, 1, 300, 280, 50), ret(300, 400, (0.98, 0.9)), 130), layer(heads(70, 2, 16, 16, 33), ret(64, 300, (0.9, 0.99)), 64)], side=130)
# one wide group: 34 query heads on one key head (two row blocks of the split kernel), chunks of one and two positions
GROUPS = config(128, 77, [layer(heads(34, 1, 32, 32, 1), ret(32, 32, (0.9, 0.97)), 64), layer(heads(34, 1, 32, 32, 2), ret(32, 32, (0.95, 0.99)), 64), layer(heads(37, 1, 16, 16, 500), ret(64, 64, (0.999,)), 64)],
                side=8, loop=(2, 3, 2))
# the smallest of everything
TINY = config(64, 40, [layer(heads(1, 1, 16, 16, 8, rot=(100.0, 2)), ret(16, 16, (0.9,), rot=(100.0, 0)), 16)], side=4, loop=(0, 1, 1))


def weights(cfg, seed=0, qk_gain=1.0, out_gain=1.0):
    """bf16 weights under the checkpoint's names.  qk_gain > 1 sharpens every attention (scores of a few units: a wrong key shows)."""
    from callireader_amd.config import DecoderSpec
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in DecoderSpec.from_lugasun(cfg).weight_shapes().items():
        r = torch.randn(*shape, generator=g)
        leaf = name.rsplit('.', 1)[-1]
        if name == 'embed':
            t = out_gain * r
        elif name == 'side.embed':
            t = 2.0 * r
        elif leaf.startswith('norm'):
            t = 1.0 + 0.3 * r
            if name.endswith('q.norm'):
                t = qk_gain * t
            if name == 'final.norm':
                t = t / math.sqrt(cfg['width'])
        else:
            t = r / math.sqrt(shape[1])
        out[name] = t.to(torch.bfloat16)
    return out


def tokens(cfg, n, seed=0):
    return torch.randint(0, cfg['vocab'], (n,), generator=torch.Generator().manual_seed(1000 + seed)).tolist()


def rel(a, b):
    """Largest row error: rms of the difference over the rms of the reference (mean of a row taken off)."""
    d = (a - b).float()
    d = d - d.mean(-1, keepdim=True)
    return float((d.pow(2).mean(-1).sqrt() / b.float().std()).max())


def close(a, b, dtype):
    """float32: rounding of sums alone (2e-5).  bfloat16: a token whose retention scores nearly cancel is divided by nearly nothing, so single rows may carry several times the usual
    rounding; half of all rows stay below 2e-2 of the reference's spread and every row below 1e-1."""
    if dtype == torch.float32:
        return rel(a, b) < 2e-5
    d = (a - b).float()
    d = (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / b.float().std()
    return float(d.median()) < 2e-2 and float(d.max()) < 1e-1
