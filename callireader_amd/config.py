"""Shapes of the CalliReader image->text hot path.

Every number here comes from the reference's HF config, not from us:
  /root/reference/InternVL/config.json:11      downsample_ratio 0.5
  /root/reference/InternVL/config.json:14-103  llm_config  (InternLM2.5-7B)
  /root/reference/InternVL/config.json:114-143 vision_config (InternViT-300M)
  /root/reference/InternVL/modeling_internvl_chat.py:157  resampler depth 4
  /root/reference/models/perceiver_resampler.py:54-64     resampler dim_head 64, heads 8, 3 queries, ff x4

`ModelDims.full()` is the checkpoint's shape; `ModelDims.reduced()` keeps every
width but cuts depths so that the CPU oracle finishes in seconds (parity tests).
"""
from dataclasses import dataclass, asdict, replace

IMG_CONTEXT_TOKEN_ID = 92546   # '<IMG_CONTEXT>'  (reference added_tokens.json)
ALIGNED_TOKEN_ID = 92537       # '[UNUSED_TOKEN_140]' (modeling_internvl_chat.py:1100)
EOS_TOKEN_ID = 92542           # '<|im_end|>'     (modeling_internvl_chat.py:709,732)


@dataclass(frozen=True)
class ModelDims:
    # InternViT-300M
    image_size: int = 448
    patch_size: int = 14
    vit_hidden: int = 1024
    vit_heads: int = 16
    vit_ff: int = 4096
    vit_layers: int = 24
    vit_ln_eps: float = 1e-6
    # projector (pixel-shuffle 0.5 + mlp1)
    downsample_ratio: float = 0.5
    # PerceiverResampler ("CalliAlign")
    rs_depth: int = 4
    rs_heads: int = 8
    rs_dim_head: int = 64
    rs_queries: int = 3
    rs_ff_mult: int = 4
    # InternLM2.5-7B
    llm_hidden: int = 4096
    llm_heads: int = 32
    llm_kv_heads: int = 8
    llm_ff: int = 14336
    llm_layers: int = 32
    vocab: int = 92553
    rms_eps: float = 1e-5
    rope_theta: float = 1000000.0
    rope_factor: float = 2.0
    max_pos: int = 32768

    @property
    def n_patches(self):
        return (self.image_size // self.patch_size) ** 2          # 1024

    @property
    def vit_tokens(self):
        return self.n_patches + 1                                 # 1025

    @property
    def vit_head_dim(self):
        return self.vit_hidden // self.vit_heads                  # 64

    @property
    def tokens_per_tile(self):
        return int(self.n_patches * self.downsample_ratio ** 2)   # 256

    @property
    def proj_in(self):
        return self.vit_hidden * int(1 / self.downsample_ratio) ** 2   # 4096

    @property
    def llm_head_dim(self):
        return self.llm_hidden // self.llm_heads                  # 128

    @property
    def rs_inner(self):
        return self.rs_heads * self.rs_dim_head                   # 512

    @staticmethod
    def full():
        return ModelDims()

    @staticmethod
    def reduced(vit_layers=2, llm_layers=2, rs_depth=2, vocab=None):
        d = ModelDims()
        kw = dict(vit_layers=vit_layers, llm_layers=llm_layers, rs_depth=rs_depth)
        if vocab is not None:
            kw['vocab'] = vocab
        return replace(d, **kw)

    @staticmethod
    def from_hf_config(path, rs_depth=None):
        """Shapes from a checkpoint directory's config.json (the file AutoModel.from_pretrained reads,
        /root/reference/inference.py:85-89): depths, vocabulary, eps, RoPE base; widths must be the path's own (the HIP
        kernels are built for InternViT-300M / InternLM2.5-7B widths).  The resampler depth is not in config.json
        (modeling_internvl_chat.py:157 hard-codes 4): pass `rs_depth` or it is read off the checkpoint's key names."""
        import json
        import os
        with open(os.path.join(path, 'config.json')) as f:
            cfg = json.load(f)
        v, l = cfg['vision_config'], cfg['llm_config']
        d = ModelDims()
        want = dict(vit_hidden=v['hidden_size'], vit_heads=v['num_attention_heads'], vit_ff=v['intermediate_size'],
                    image_size=v['image_size'], patch_size=v['patch_size'], llm_hidden=l['hidden_size'],
                    llm_heads=l['num_attention_heads'], llm_kv_heads=l['num_key_value_heads'], llm_ff=l['intermediate_size'])
        for k, val in want.items():
            if getattr(d, k) != val:
                raise ValueError(f'config.json {k}={val}: this engine is built for {k}={getattr(d, k)}')
        if rs_depth is None:
            rs_depth = d.rs_depth
            idx = os.path.join(path, 'model.safetensors.index.json')
            if os.path.exists(idx):
                with open(idx) as f:
                    keys = json.load(f)['weight_map'].keys()
                layers = {int(k.split('.')[2]) for k in keys if k.startswith('resampler.layers.')}
                if layers:
                    rs_depth = max(layers) + 1
        rope = l.get('rope_scaling') or {}
        return replace(d, vit_layers=v['num_hidden_layers'], llm_layers=l['num_hidden_layers'], vocab=l['vocab_size'],
                       vit_ln_eps=v.get('layer_norm_eps', d.vit_ln_eps), rms_eps=l.get('rms_norm_eps', d.rms_eps),
                       rope_theta=float(l.get('rope_theta', d.rope_theta)), rope_factor=float(rope.get('factor', d.rope_factor)),
                       max_pos=l.get('max_position_embeddings', d.max_pos), downsample_ratio=cfg.get('downsample_ratio', d.downsample_ratio),
                       rs_depth=rs_depth)

    def asdict(self):
        return asdict(self)


# ---- described decoders: language models whose layers are read from config.json ----------------------------------------------

@dataclass(frozen=True)
class LatentMixer:
    """Latent attention (include/callireader_hip.h: CR_MIX_LATENT)."""
    heads: int
    dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float

    def weight_shapes(self, p, W):
        return {p + 'dq': (self.q_rank, W), p + 'dq.norm': (self.q_rank,), p + 'uq': (self.heads * self.dim, self.q_rank), p + 'dkv': (self.kv_rank, W), p + 'dkv.norm': (self.kv_rank,),
                p + 'uk': (self.heads * self.dim, self.kv_rank), p + 'uv': (self.heads * self.vdim, self.kv_rank), p + 'g': (self.heads * self.vdim, W),
                p + 'o': (W, self.heads * self.vdim)}


@dataclass(frozen=True)
class Rotation:
    """Entries i and i + dims / 2 of a head turn by position * base^(-2 i / dims); entries from `dims` on stay."""
    base: float
    dims: int


@dataclass(frozen=True)
class HeadsMixer:
    """Softmax attention over grouped heads (CR_MIX_HEADS); chunk: keys of the query's own chunk of positions only (0: every earlier key)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Rotation = None
    chunk: int = 0
    softcap: float = 0.0
    qk_norm: bool = False

    def weight_shapes(self, p, W):
        out = {p + 'q': (self.heads * self.dim, W), p + 'k': (self.kv_heads * self.dim, W), p + 'v': (self.kv_heads * self.vdim, W), p + 'o': (W, self.heads * self.vdim)}
        return {**out, p + 'q.norm': (self.dim,), p + 'k.norm': (self.dim,)} if self.qk_norm else out


@dataclass(frozen=True)
class RetentionMixer:
    """Linear attention with a fixed decay per head (CR_MIX_RETENTION)."""
    heads: int
    dim: int
    vdim: int
    decay: tuple
    k_scale: float
    rot: Rotation = None

    def weight_shapes(self, p, W):
        return {p + 'q': (self.heads * self.dim, W), p + 'k': (self.heads * self.dim, W), p + 'v': (self.heads * self.vdim, W), p + 'g': (self.heads * self.vdim, W),
                p + 'o': (W, self.heads * self.vdim)}


@dataclass(frozen=True)
class ParallelMixer:
    """Attention and retention on the same input, outputs added: left_scale * left + right_scale * right."""
    left: HeadsMixer
    right: RetentionMixer
    left_scale: float = 1.0
    right_scale: float = 1.0

    def weight_shapes(self, p, W):
        return {**self.left.weight_shapes(p + 'left.', W), **self.right.weight_shapes(p + 'right.', W)}


@dataclass(frozen=True)
class ExpertMixture:
    """Clamped gated experts behind a grouped router (CR_FF_MOE)."""
    experts: int
    top: int
    ff: int
    limit: float
    groups: int = 1
    keep: int = 1

    def weight_shapes(self, p, W):
        out = {p + 'router': (self.experts, W), p + 'correction': (self.experts,)}
        for e in range(self.experts):
            out.update({f'{p}e{e}.gate': (self.ff, W), f'{p}e{e}.up': (self.ff, W), f'{p}e{e}.down': (W, self.ff)})
        return out


@dataclass(frozen=True)
class DenseFF:
    """W_down act(W_up h) (CR_FF_DENSE)."""
    ff: int
    act: str = 'relu2'

    def weight_shapes(self, p, W):
        return {p + 'up': (self.ff, W), p + 'down': (W, self.ff)}


@dataclass(frozen=True)
class DecoderLayer:
    mixer: object                    # LatentMixer, HeadsMixer, RetentionMixer or ParallelMixer
    ff: object = None                # ExpertMixture, DenseFF or none


@dataclass(frozen=True)
class DecoderSpec:
    """A decoder-only model as the engine runs it: sizes, constants and the order of layers (one weight set per entry of `layers`)."""
    width: int
    vocab: int
    layers: tuple
    eps: float
    loop: tuple = None               # (start, stop, times): layers [start, stop) run `times` times in a row
    softcap: float = 0.0             # 0: no cap on the logits
    sinusoid_base: float = 0.0       # > 0: a sinusoidal position vector is added to the embedding
    norm_plain: bool = False         # the model's norms multiply by their weight (otherwise by one plus their weight)
    post_norm: bool = True           # a sublayer's output goes through a norm of its own before it joins the residual
    tied_head: bool = False          # logits from the embedding table
    loop_in: bool = False            # x <- W [x; embedding] ahead of every pass of the looped span
    side_dim: int = 0                # > 0: per-layer token input of this width after the feed-forward

    @property
    def passes(self):
        """Layer index of every layer pass, the looped span unrolled."""
        n = len(self.layers)
        if not self.loop:
            return list(range(n))
        a, z, t = self.loop
        return list(range(a)) + list(range(a, z)) * t + list(range(z, n))

    def weight_shapes(self):
        """name -> shape of every checkpoint tensor."""
        W, out = self.width, {'embed': (self.vocab, self.width), 'final.norm': (self.width,)}
        if not self.tied_head:
            out['head'] = (self.vocab, W)
        if self.loop_in and self.loop:
            out['loop.in'] = (W, 2 * W)
        if self.side_dim:
            out['side.embed'] = (self.vocab, len(self.layers) * self.side_dim)
        for i, layer in enumerate(self.layers):
            p = f'l{i}.'
            for j, sub in enumerate((layer.mixer, layer.ff), 1):
                if sub is None:
                    continue
                out[f'{p}norm{j}'] = (W,)
                if self.post_norm:
                    out[f'{p}norm{j}b'] = (W,)
                out.update(sub.weight_shapes(p + ('mix.' if j == 1 else 'mlp.'), W))
            if self.side_dim:
                out.update({p + 'side.gate': (self.side_dim, W), p + 'side.proj': (W, self.side_dim), p + 'side.norm': (W,)})
        return out

    @staticmethod
    def from_linasun(cfg):
        """The Linasun design's config.json (parsed)."""
        layers = []
        for i, entry in enumerate(cfg['layers']):
            if entry['type'] != 'latent_attention':
                raise ValueError(f'layer {i}: unknown mixer {entry["type"]!r}')
            m = entry['mixer']
            mixer = LatentMixer(heads=m['heads'], dim=m['dim'], vdim=m['vdim'], q_rank=m['q_rank'], kv_rank=m['kv_rank'], scale=float(m['scale']))
            ff, mlp = None, entry.get('mlp')
            if mlp is not None:
                if mlp.get('kind', 'moe') != 'moe':
                    raise ValueError(f'layer {i}: unknown feed-forward {mlp["kind"]!r}')
                r, g = mlp['router'], mlp['router'].get('groups') or {'count': 1, 'keep': 1}
                ff = ExpertMixture(experts=r['experts'], top=r['top'], ff=mlp['expert']['ff'], limit=float(mlp['expert']['limit']), groups=g['count'], keep=g['keep'])
            layers.append(DecoderLayer(mixer, ff))
        lp = cfg.get('loop')
        return DecoderSpec(width=cfg['width'], vocab=cfg['vocab'], layers=tuple(layers), eps=float(cfg['norm']['eps']),
                           loop=(lp['start'], lp['stop'], lp['times']) if lp else None, softcap=float(cfg.get('logit_softcap') or 0.0), sinusoid_base=10000.0)

    @staticmethod
    def from_lugasun(cfg):
        """The Lugasun design's config.json (parsed)."""
        def rotation(m):
            r = m.get('rot')
            return Rotation(base=float(r['base']), dims=r['dims']) if r and r['dims'] else None
        layers = []
        for i, entry in enumerate(cfg['layers']):
            if entry['type'] != 'parallel':
                raise ValueError(f'layer {i}: unknown mixer {entry["type"]!r}')
            m = entry['mixer']
            a, r = m['left'], m['right']
            left = HeadsMixer(heads=a['heads'], kv_heads=a['kv_heads'], dim=a['dim'], vdim=a['vdim'], scale=float(a['scale']), rot=rotation(a),
                              chunk=(a.get('mask') or {}).get('size') or 0, softcap=float(a.get('softcap') or 0.0), qk_norm=True)
            if len(r['decay']) != r['heads']:
                raise ValueError(f'layer {i}: {len(r["decay"])} decays for {r["heads"]} heads')
            right = RetentionMixer(heads=r['heads'], dim=r['dim'], vdim=r['vdim'], decay=tuple(float(d) for d in r['decay']), k_scale=r['dim'] ** -0.5, rot=rotation(r))
            mlp = entry.get('mlp')
            if mlp is not None and mlp['kind'] != 'dense':
                raise ValueError(f'layer {i}: unknown feed-forward {mlp["kind"]!r}')
            layers.append(DecoderLayer(ParallelMixer(left, right, float(m['left_scale']), float(m['right_scale'])), DenseFF(mlp['ff']) if mlp is not None else None))
        lp, side = cfg.get('loop'), cfg.get('token_side')
        return DecoderSpec(width=cfg['width'], vocab=cfg['vocab'], layers=tuple(layers), eps=float(cfg['norm']['eps']), loop=(lp['start'], lp['stop'], lp['times']) if lp else None,
                           norm_plain=True, post_norm=False, tied_head=True, loop_in=bool(lp), side_dim=side['dim'] if side else 0)
