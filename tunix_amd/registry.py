"""Model registry: config.json of a model folder -> configuration and device-resident model.

A folder holds config.json and *.safetensors.  The architecture named by config.json ('architecture', or the first
entry of 'architectures') picks the entry; every model the registry returns runs behind the same Sampler.
"""
import glob
import json
import os
from typing import Callable, NamedTuple

import torch

from tunix_amd import checkpoint
from tunix_amd.grouped import GroupedConfig, GroupedModel
from tunix_amd.latent import LatentConfig, LatentModel
from tunix_amd.model import ModelConfig


class Entry(NamedTuple):
  dtypes: tuple         # activation formats the model runs in
  config: Callable      # (mapping, dtype) -> configuration
  load: Callable        # (folder, configuration, device, **options) -> model


def read_config(folder):
  with open(os.path.join(folder, 'config.json')) as f:
    return json.load(f)


def read_tensors(folder):
  """Every tensor of every *.safetensors file under the folder, on the CPU."""
  from safetensors import safe_open
  files = sorted(glob.glob(os.path.join(folder, '*.safetensors')))
  if not files:
    raise FileNotFoundError(f'no *.safetensors under {folder}')
  out = {}
  for path in files:
    with safe_open(path, framework='pt', device='cpu') as sf:
      for k in sf.keys():
        out[k] = sf.get_tensor(k)
  return out


def _load_dense(model):
  return lambda folder, config, device: model.from_state(config, read_tensors(folder), device=device)


def _hf_config(family):
  def parse(cfg, dtype):
    del dtype
    heads = int(cfg['num_attention_heads'])
    rope = cfg.get('rope_theta', (cfg.get('rope_parameters') or {}).get('rope_theta', 10_000.0))
    experts = cfg.get('num_experts')
    return ModelConfig(family, int(cfg['num_hidden_layers']), int(cfg['vocab_size']), int(cfg['hidden_size']),
                       int(cfg['moe_intermediate_size'] if experts else cfg['intermediate_size']), heads,
                       int(cfg.get('head_dim') or cfg['hidden_size'] // heads), int(cfg.get('num_key_value_heads') or heads),
                       float(rope), float(cfg.get('rms_norm_eps', 1e-6)), bool(cfg.get('tie_word_embeddings', False)),
                       experts, cfg.get('num_experts_per_tok') if experts else None)
  return parse


def _load_quantised(folder, config, device, **options):
  return checkpoint.model_from_hf(folder, config, device=device, **options)


ARCHITECTURES = {
    'Feduzen': Entry(('bfloat16', 'float32'), GroupedConfig.from_dict, _load_dense(GroupedModel)),
    'Kagapel': Entry(('bfloat16', 'float32'), LatentConfig.from_dict, _load_dense(LatentModel)),
    'LlamaForCausalLM': Entry(('bfloat16',), _hf_config('llama3'), _load_quantised),
    'Qwen3ForCausalLM': Entry(('bfloat16',), _hf_config('qwen3'), _load_quantised),
    'Qwen3MoeForCausalLM': Entry(('bfloat16',), _hf_config('qwen3'), _load_quantised),
}


def entry_of(cfg):
  name = cfg.get('architecture') or (cfg.get('architectures') or [None])[0]
  if name not in ARCHITECTURES:
    raise ValueError(f'unknown architecture {name!r} (known: {sorted(ARCHITECTURES)})')
  return ARCHITECTURES[name]


def load_config(folder, dtype='bfloat16'):
  cfg = read_config(folder)
  entry = entry_of(cfg)
  if dtype not in entry.dtypes:
    raise ValueError(f'this architecture runs in {", ".join(entry.dtypes)}, not in {dtype}')
  return entry.config(cfg, dtype)


def load_model(folder, dtype='bfloat16', device='cuda', **options):
  config = load_config(folder, dtype)
  with torch.no_grad():
    return entry_of(read_config(folder)).load(folder, config, device, **options)
