"""Which class serves a checkpoint directory: decided by its config.json."""
import importlib
import json
import os

# architecture name in config.json ('architecture', or the HF list 'architectures') -> (module, class)
MODELS = {
    'InternVLChatModel': ('.modeling_internvl_chat', 'InternVLChatModel'),
    'Linasun': ('.modeling_decoder', 'LinasunForCausalLM'),
    'Lugasun': ('.modeling_decoder', 'LugasunForCausalLM'),
}
DEFAULT = 'InternVLChatModel'            # the reference's checkpoints, and directories without a config.json


def architecture(path):
    f = os.path.join(path, 'config.json')
    if not os.path.exists(f):
        return DEFAULT
    with open(f) as fh:
        cfg = json.load(fh)
    for name in [cfg.get('architecture')] + list(cfg.get('architectures') or []):
        if name in MODELS:
            return name
    if cfg.get('architecture'):
        raise ValueError(f'{f}: unknown architecture {cfg["architecture"]!r} (known: {", ".join(sorted(MODELS))})')
    return DEFAULT


def model_class(path):
    module, name = MODELS[architecture(path)]
    return getattr(importlib.import_module(module, __package__), name)


def is_text_model(path):
    """Token ids in, token ids out (no images, no tokenizer of its own)."""
    return MODELS[architecture(path)][0] == '.modeling_decoder'
