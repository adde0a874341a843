"""`bench.py --workload linasun | lugasun`: prefill and decode throughput of a described decoder at a few sizes that resemble a real model's layers, random weights, beside the
engine's InternLM2 layers at equal width and equal (active) feed-forward weights.  One process, one GPU; HIP events on the current stream; prints one JSON line."""
import json
import math

import torch

from .measure import PEAK_BF16_TFLOPS, PEAK_HBM_GBS

PROMPTS, PROMPT, CTX = 4, 2048, 3072             # prefill: PROMPTS x PROMPT rows in one call; decode: CTX cached tokens per row
ROWS = (1, 8, 64)


def _cfg(width, heads, dim, q_rank, kv_rank, experts, top, ff, groups, layers, vocab, loop=None):
    layer = dict(type='latent_attention', mixer=dict(heads=heads, dim=dim, vdim=dim, q_rank=q_rank, kv_rank=kv_rank, scale=dim ** -0.5),
                 mlp=dict(kind='moe', expert=dict(ff=ff, limit=7.0), router=dict(experts=experts, top=top, groups=dict(count=groups[0], keep=groups[1]))))
    return dict(architecture='Linasun', width=width, vocab=vocab, norm=dict(eps=1e-6), logit_softcap=30.0, layers=[layer] * layers,
                **({'loop': dict(start=loop[0], stop=loop[1], times=loop[2])} if loop else {}))


LINASUN = {
    'w4096_e64': _cfg(4096, 32, 128, 1536, 512, 64, 8, 1792, (8, 4), 4, 92553),          # active feed-forward width 8 x 1792 = InternLM2.5-7B's 14336
    'w2048_e32': _cfg(2048, 16, 128, 768, 512, 32, 4, 1024, (4, 2), 8, 32000),
    'w1024_looped': _cfg(1024, 8, 128, 384, 256, 16, 2, 1024, (4, 2), 6, 32000, loop=(1, 5, 3)),
}


def _lugasun(width, heads, kv_heads, dim, chunk, ret_heads, ret_dim, ret_vdim, ff, side, layers, vocab, loop=None):
    left = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, mask=dict(size=chunk), scale=dim ** -0.5, softcap=50.0, rot=dict(base=1e6, dims=dim))
    right = dict(heads=ret_heads, dim=ret_dim, vdim=ret_vdim, decay=[1.0 - 2.0 ** (-5 - 6 * i / ret_heads) for i in range(ret_heads)], rot=dict(base=1e4, dims=ret_dim))
    layer = dict(type='parallel', mixer=dict(left=left, right=right, left_scale=0.7, right_scale=0.7), mlp=dict(kind='dense', ff=ff))
    return dict(architecture='Lugasun', width=width, vocab=vocab, norm=dict(eps=1e-6), layers=[layer] * layers, token_side=dict(dim=side),
                **({'loop': dict(start=loop[0], stop=loop[1], times=loop[2])} if loop else {}))


LUGASUN = {
    # attention heads, cached keys and feed-forward weights (2 x 21504 rows against 3 x 14336) are InternLM2.5-7B's; retention and the token side come on top
    'w4096_c8192': _lugasun(4096, 32, 8, 128, 8192, 32, 128, 128, 21504, 256, 4, 92553),
    'w2048_c1024': _lugasun(2048, 16, 4, 128, 1024, 8, 128, 256, 8192, 128, 8, 32000),
    'w1024_looped': _lugasun(1024, 8, 2, 128, 512, 8, 64, 64, 4096, 64, 6, 32000, loop=(1, 5, 3)),
}
SIZES = {'linasun': LINASUN, 'lugasun': LUGASUN}


def random_weights(spec, device, seed=0):
    """name, bf16 tensor: drawn on the device one by one."""
    g = torch.Generator(device=device).manual_seed(seed)
    for name, shape in spec.weight_shapes().items():
        leaf = name.rsplit('.', 1)[-1]
        r = torch.randn(*shape, device=device, generator=g)
        if len(shape) == 1:
            r = 1.0 + 0.1 * r if spec.norm_plain or (leaf == 'norm' and name != 'final.norm') else (1e-3 if leaf == 'correction' else 0.1) * r      # (small corrections: balanced experts)
        elif name != 'embed':
            r = r / math.sqrt(shape[1])
        yield name, r.to(torch.bfloat16)


def build(cfg, max_tokens, rows, device=0, dtype=torch.bfloat16):
    from callireader_amd import modeling_decoder, registry
    cls = getattr(modeling_decoder, registry.MODELS[cfg['architecture']][1])
    spec = cls.read_config(cfg)
    return cls.from_state_dict(random_weights(spec, torch.device('cuda', device)), spec, device=device, dtype=dtype, max_tokens=max_tokens, max_seqs=rows)


def _visible(n, chunk):
    """Keys that positions 0 .. n - 1 see, in all."""
    full, rest = divmod(n, chunk) if chunk else (0, n)
    return full * chunk * (chunk + 1) / 2 + rest * (rest + 1) / 2


def _mixers(m):
    from callireader_amd.config import ParallelMixer
    return [m.left, m.right] if isinstance(m, ParallelMixer) else [m]


def _ff_weights(spec, f, rows=None):
    """Feed-forward weights a token multiplies (rows=None), or that a batch of `rows` tokens reads (every expert some row is expected to choose, uniform choices)."""
    from callireader_amd.config import DenseFF
    if f is None:
        return 0
    if isinstance(f, DenseFF):
        return 2 * spec.width * f.ff
    return spec.width * f.experts + (f.top if rows is None else f.experts * (1 - (1 - f.top / f.experts) ** rows)) * 3 * spec.width * f.ff


def _mixer_weights(spec, m):
    from callireader_amd.config import HeadsMixer, RetentionMixer
    if isinstance(m, HeadsMixer):
        return spec.width * (m.heads * (m.dim + m.vdim) + m.kv_heads * (m.dim + m.vdim))
    if isinstance(m, RetentionMixer):
        return spec.width * m.heads * (2 * m.dim + 3 * m.vdim)
    return spec.width * (m.q_rank + m.kv_rank + 2 * m.heads * m.vdim) + m.q_rank * m.heads * m.dim + m.kv_rank * m.heads * (m.dim + m.vdim)


def _loop_weights(spec):
    return (spec.loop[2] if spec.loop_in and spec.loop else 0) * 2 * spec.width * spec.width


def prefill_flops(spec, tokens, seqs):
    """2 x multiply-adds of the equations as written (keys and values formed once per token, retention as its recurrence), visible keys of the attention, logits of the last rows."""
    from callireader_amd.config import HeadsMixer, RetentionMixer
    f = 2.0 * tokens * _loop_weights(spec)
    for i in spec.passes:
        for m in _mixers(spec.layers[i].mixer):
            f += 2.0 * tokens * _mixer_weights(spec, m)
            if isinstance(m, RetentionMixer):
                f += 2.0 * tokens * m.heads * 2 * m.dim * m.vdim
            else:
                f += 2.0 * seqs * _visible(tokens // seqs, m.chunk if isinstance(m, HeadsMixer) else 0) * m.heads * (m.dim + m.vdim)
        f += 2.0 * tokens * (_ff_weights(spec, spec.layers[i].ff) + 2 * spec.width * spec.side_dim)
    return f + 2.0 * seqs * spec.width * spec.vocab


def decode_bytes(spec, rows, ctx):
    """Weights and cache a decode step has to read once, and the states it reads and writes."""
    from callireader_amd.config import HeadsMixer, RetentionMixer
    b = 2.0 * spec.width * spec.vocab + 2.0 * _loop_weights(spec)
    for i in spec.passes:
        for m in _mixers(spec.layers[i].mixer):
            b += 2.0 * _mixer_weights(spec, m)
            if isinstance(m, RetentionMixer):
                b += 8.0 * rows * m.heads * m.dim * m.vdim
            elif isinstance(m, HeadsMixer):
                b += 2.0 * rows * (ctx % m.chunk + 1 if m.chunk else ctx) * m.kv_heads * (m.dim + m.vdim)
            else:
                b += 2.0 * rows * ctx * m.kv_rank
        b += 2.0 * (_ff_weights(spec, spec.layers[i].ff, rows) + 2 * spec.width * spec.side_dim)
    return b


def timed(fn, reps):
    a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    fn()
    torch.cuda.synchronize()
    a.record()
    for _ in range(reps):
        fn()
    b.record()
    torch.cuda.synchronize()
    return a.elapsed_time(b) / reps


def measure(kv, prefill, decode, flops, bytes_of, steps=20):
    """prefill(): fills the first PROMPTS sequences; decode(rows): one step."""
    def pre():
        kv.reset()
        prefill(list(range(PROMPTS)), PROMPT)
    ms = timed(pre, 3)
    out = {'prefill': {'rows': f'{PROMPTS} x {PROMPT}', 'ms': round(ms, 3), 'tokens_per_s': round(PROMPTS * PROMPT / ms * 1e3), 'tflops': round(flops / ms / 1e9, 1),
                       'mfma_frac': round(flops / ms / 1e9 / PEAK_BF16_TFLOPS, 4)}, 'decode': {}}
    kv.reset()
    for s in range(0, max(ROWS), 4):
        prefill(list(range(s, min(s + 4, max(ROWS)))), CTX)
    for rows in ROWS:
        ms = timed(lambda: decode(list(range(rows))), steps)
        gb = bytes_of(rows) / 1e9
        out['decode'][str(rows)] = {'ctx': CTX, 'ms': round(ms, 4), 'tokens_per_s': round(rows / ms * 1e3, 1), 'gb': round(gb, 3), 'gb_per_s': round(gb / ms * 1e3, 1),
                                    'hbm_frac': round(gb / ms * 1e3 / PEAK_HBM_GBS, 4)}
    return out


def run_size(workload, name, dev):
    m = build(SIZES[workload][name], CTX + 3 * 25, max(ROWS), dev.index)
    e, spec = m.engine, m.spec
    kv = e.kv_alloc(max(ROWS), CTX + 3 * 25)
    g = torch.Generator().manual_seed(1)
    toks = torch.randint(0, spec.vocab, (max(ROWS), max(PROMPT, CTX)), generator=g).tolist()       # every row its own tokens: its own experts
    step_ids = torch.randperm(spec.vocab, generator=g)[:max(ROWS)].to(dev)                       # ... in decoding too
    out = measure(kv, lambda seqs, n: e.prefill_tokens(kv, seqs, [toks[s][:n] for s in seqs]), lambda rows: e.decode(kv, rows, force_tokens=step_ids[:len(rows)]),
                  prefill_flops(spec, PROMPTS * PROMPT, PROMPTS), lambda rows: decode_bytes(spec, rows, CTX))
    out['layer_passes'] = len(spec.passes)
    kv.free()
    m.close()
    return out


def run_internlm2(dev, layers=4):
    """The engine's own language model, `layers` layers of InternLM2.5-7B (width 4096, 32 query / 8 KV heads x 128, feed-forward 14336) with its vocabulary."""
    from callireader_amd.config import ModelDims
    from callireader_amd.modeling_internvl_chat import InternVLChatModel
    dims = ModelDims.reduced(vit_layers=0, llm_layers=layers, rs_depth=0)
    m = InternVLChatModel.from_synthetic(dims, seed=0, parts=('llm',), device=dev.index, max_tokens=CTX + 3 * 25, max_pages=max(ROWS))
    e = m.engine
    kv = e.kv_alloc(max(ROWS), CTX + 3 * 25)
    emb = (torch.randn(4 * max(PROMPT, CTX), dims.llm_hidden, device=dev) * 0.02).bfloat16()
    lin = layers * (4096 * 6144 + 4096 * 4096 + 3 * 4096 * 14336)
    t = PROMPTS * PROMPT
    # what its prefill computes: the last layer's attention, wo and feed-forward run on the last rows only
    done = lin - (4096 * 4096 + 3 * 4096 * 14336)
    flops = 2.0 * t * done + (layers - 1) * 4.0 * PROMPTS * PROMPT * (PROMPT + 1) / 2 * 4096 + 2.0 * PROMPTS * 4096 * dims.vocab
    out = measure(kv, lambda seqs, n: e.prefill_batch(kv, seqs, [emb[i * n:(i + 1) * n] for i in range(len(seqs))]), lambda rows: e.decode(kv, rows), flops,
                  lambda rows: 2.0 * (lin + 4096 * dims.vocab) + layers * rows * CTX * 2 * 8 * 128 * 2)
    out['layer_passes'] = layers
    kv.free()
    m.close()
    return out


def _describe(workload, c):
    layer = c['layers'][0]
    d = dict(width=c['width'], layers=len(c['layers']), loop=c.get('loop'), vocab=c['vocab'])
    if workload == 'lugasun':
        left, right = layer['mixer']['left'], {k: v for k, v in layer['mixer']['right'].items() if k not in ('decay', 'rot')}
        return dict(d, attention={k: v for k, v in left.items() if k not in ('rot', 'mask')}, chunk=left['mask']['size'], retention=right, ff=layer['mlp']['ff'], token_side=c['token_side']['dim'])
    return dict(d, **layer['mixer'], experts=layer['mlp']['router']['experts'], top=layer['mlp']['router']['top'], expert_ff=layer['mlp']['expert']['ff'])


def run(workload, dev, only=None):
    res = {}
    with torch.inference_mode():
        if not only or 'internlm2' in only:
            res['internlm2_4_layers'] = run_internlm2(dev)
        for name in SIZES[workload]:
            if not only or name in only:
                res[name] = run_size(workload, name, dev)
                torch.cuda.empty_cache()
    ref = res.get(next(iter(SIZES[workload]))) or next(v for k, v in res.items())
    return {'metric': f'{workload.capitalize()} layers: decode tokens/s (64 rows, 4 layers of width 4096)', 'value': ref['decode']['64']['tokens_per_s'], 'unit': 'tokens/s', 'n_gpus': 1,
            'higher_is_better': True, 'vs_baseline': None, 'dtype': 'bf16', 'data': 'synthetic', 'sizes': res, 'config': {k: _describe(workload, c) for k, c in SIZES[workload].items()},
            'how': 'HIP events around whole engine calls after a warm-up call; flops and bytes are algorithmic (this file), peaks as everywhere in bench.py'}


def main(workload, dev, only=None):
    print(json.dumps(run(workload, dev, only)), flush=True)
