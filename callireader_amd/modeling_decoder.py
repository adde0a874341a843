"""Described decoders as models: token ids in, token ids (or logits) out, over the engine's cache, batched greedy loop and kernels.

A design is a reader of its config.json (config.DecoderSpec.from_*), listed in registry.py; everything below is shared by all of them.
"""
import json
import os

import torch

from .batching import SequenceSlots, decode_greedy
from .config import DecoderSpec
from .engine import DecoderEngine


class DecoderLM:
    main_input_name = 'input_ids'
    read_config = None               # config.json (parsed) -> DecoderSpec

    def __init__(self, spec, dtype=torch.bfloat16, device=0, max_tokens=8192, max_seqs=1):
        self.spec, self.max_tokens = spec, max_tokens
        self.engine = DecoderEngine(spec, dtype=dtype, device=device)
        self.device = self.engine.device
        self.slots = SequenceSlots(self.engine, max_tokens, max_seqs)

    # ---- construction --------------------------------------------------------------------------
    @classmethod
    def from_state_dict(cls, sd, config, **kw):
        m = cls(config if isinstance(config, DecoderSpec) else cls.read_config(config), **kw)
        m._load(sd.items() if hasattr(sd, 'items') else sd)
        return m

    @classmethod
    def from_pretrained(cls, path, dtype=torch.bfloat16, **kw):
        from .weights import iter_safetensors
        with open(os.path.join(path, 'config.json')) as f:
            spec = cls.read_config(json.load(f))
        m = cls(spec, dtype=dtype, **kw)
        m._load(iter_safetensors(path))
        return m

    def _load(self, items):
        want = self.spec.weight_shapes()
        for name, t in items:
            shape = want.pop(name, None)
            if shape is None:
                continue
            if tuple(t.shape) != tuple(shape):
                raise ValueError(f'{name}: {tuple(t.shape)}, the configuration says {tuple(shape)}')
            self.engine.load_weight(name, t.to(torch.bfloat16))
        if want:
            raise KeyError(f'{len(want)} tensors missing, the first is {sorted(want)[0]}')
        self.engine.finalize()

    def eval(self):
        return self

    def cuda(self):
        return self

    def close(self):
        self.slots.close()
        self.engine.close()

    # ---- one step ------------------------------------------------------------------------------
    def step(self, entries, penalty=1.0):
        """entries: (request id, next token ids, places among them whose logits are wanted).  Runs exactly these tokens on top of what the requests have cached; unknown ids are new
        requests.  -> fp32 logits [wanted, vocab] in the order of the entries and places, or None.  One token each on top of a cache is a decode step, anything else a prefill."""
        new = [rid for rid, _, _ in entries if rid not in self.slots.slot]
        if new:
            self.slots.admit(new)
        kv = self.slots.kv
        seqs = [self.slots.slot[rid] for rid, _, _ in entries]
        if not new and all(len(t) == 1 for _, t, _ in entries):
            logits = self.engine.decode(kv, seqs, penalty=penalty, force_tokens=torch.tensor([t[0] for _, t, _ in entries], dtype=torch.int64), want_logits=True)
            rows = [i for i, (_, _, w) in enumerate(entries) for _ in w]
            return logits[rows] if rows else None
        want, base = [], 0
        for _, t, w in entries:
            want += [base + p for p in w]
            base += len(t)
        return self.engine.prefill_tokens(kv, seqs, [t for _, t, _ in entries], penalty=penalty, want=want)

    def end(self, rid):
        self.slots.release(rid)

    # ---- generation ----------------------------------------------------------------------------
    @torch.no_grad()
    def generate(self, prompts, max_new_tokens=128, eos_token_id=None, repetition_penalty=1.0, check_every=16, prefill_tokens=16384):
        """prompts: lists of token ids, decoded greedily as one batch; -> the new ids of each, EOS included."""
        prompts = [[int(t) for t in p] for p in prompts]
        if not prompts or max_new_tokens <= 0:
            return [[] for _ in prompts]
        for p in prompts:
            if not p or len(p) + max_new_tokens > self.max_tokens:
                raise ValueError(f'prompt of {len(p)} tokens + {max_new_tokens} new: between 1 and max_tokens={self.max_tokens}')
        rids = [('generate', i) for i in range(len(prompts))]
        slots = self.slots.admit(rids)
        try:
            i = 0
            while i < len(prompts):                       # prompts share the prefill's products up to `prefill_tokens` rows
                j, rows = i, 0
                while j < len(prompts) and (j == i or rows + len(prompts[j]) <= prefill_tokens):
                    rows += len(prompts[j])
                    j += 1
                self.engine.prefill_tokens(self.slots.kv, slots[i:j], prompts[i:j], penalty=repetition_penalty)
                i = j
            return decode_greedy(self.engine, self.slots.kv, slots, max_new_tokens, eos_token_id, repetition_penalty, check_every)
        finally:
            for r in rids:
                self.slots.release(r)


class LinasunForCausalLM(DecoderLM):
    """Looped latent-attention decoder with clamped expert mixtures, norms on both sides of every sublayer and soft-capped logits."""
    read_config = staticmethod(DecoderSpec.from_linasun)


class LugasunForCausalLM(DecoderLM):
    """Looped decoder whose layers run chunked attention and retention side by side, with a squared-relu feed-forward and a per-layer token input."""
    read_config = staticmethod(DecoderSpec.from_lugasun)
