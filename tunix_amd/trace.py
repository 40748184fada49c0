"""Replays a trace of token ids through a model and writes logits (command line of bin/trace_run).

Steps come from standard input, one JSON object a line:

  {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

The requests of a step are one batch: they all start, or all go on by one token.  A batch runs behind the Sampler
like a rollout does: prompts padded on the left to one length, one column of the cache per step, rows whose request
has ended walking on unread.  Per step in which something is wanted, OUT/<step>.f32 holds the logits at the wanted
places ([wanted, vocab], little-endian f32); 'done <step>' follows on standard output.
"""
import argparse
import dataclasses
import json
import os
import sys

import numpy as np


class IdTokenizer:
  """Token ids only; padding columns are masked by their lengths, so any valid id pads."""

  def encode(self, text, **kw):
    return [int(t) for t in text.split()]

  def decode(self, ids, **kw):
    return ' '.join(str(int(i)) for i in ids)

  def pad_id(self):
    return 0

  def bos_id(self):
    return 0

  def eos_id(self):
    return -1


class Replay:
  """The batches of a trace on one model, one after the other."""

  def __init__(self, model, max_tokens):
    from tunix_amd.configs import CacheConfig
    from tunix_amd.sampler import Sampler
    c = model.config
    self.model, self.max_tokens = model, max_tokens
    self.sampler = Sampler(model, IdTokenizer(), CacheConfig(1, c.num_layers, c.num_kv_heads, c.head_dim))
    self.sampler.eos_ids = np.array([-1])
    self.state, self.rows, self.lengths, self.column = None, {}, {}, 0

  def _check(self, tokens, length):
    vocab, limit = self.model.config.vocab_size, self.model.config.max_positions
    if any(not 0 <= t < vocab for t in tokens):
      raise ValueError(f'token id outside the vocabulary [0, {vocab})')
    if limit is not None and length > limit:
      raise ValueError(f'a request of {length} tokens exceeds the {limit} positions of the model')

  def _start(self, entries):
    """A new batch: prompts padded on the left, the cache sized for the longest continuation."""
    if self.rows:
      raise ValueError('requests may only join when the batch before them has ended')
    for e in entries:
      self._check(e['tokens'], len(e['tokens']))
      if not e['tokens']:
        raise ValueError('a request starts with at least one token')
    lens = [len(e['tokens']) for e in entries]
    width = max(lens)
    limit = min(self.model.config.max_positions or self.max_tokens, self.max_tokens)
    total = width + max(0, limit - min(lens)) + 1
    ids = np.zeros((len(entries), width), np.int32)
    for i, e in enumerate(entries):
      ids[i, width - lens[i]:] = e['tokens']
    self.sampler.cache_config = dataclasses.replace(self.sampler.cache_config, cache_size=total)
    self.state = self.sampler.init_sample_state(ids, total, False, None, 1.0, None, None, 0,
                                                prompt_lengths=np.array(lens))
    self.state['fresh'] = False
    self.rows = {e['id']: i for i, e in enumerate(entries)}
    self.lengths = {e['id']: n for e, n in zip(entries, lens)}
    self.column = width
    wanted = [(i, width - lens[i] + w) for i, e in enumerate(entries) for w in e['want']]
    return self.sampler.walk_logits(self.state, width, wanted)

  def _go_on(self, entries):
    """One known token for every entry; rows without an entry repeat the padding id."""
    import torch
    b = self.state['token_buffer'].shape[0]
    if self.column >= self.sampler.cache_config.cache_size:
      raise ValueError('the batch holds more tokens than announced')
    col = np.zeros(b, np.int32)
    for e in entries:
      if len(e['tokens']) != 1:
        raise ValueError('a running request goes on by one token')
      self.lengths[e['id']] += 1
      self._check(e['tokens'], self.lengths[e['id']])
      col[self.rows[e['id']]] = e['tokens'][0]
    self.state['token_buffer'][:, self.column] = torch.from_numpy(col).to(self.model.device)
    self.column += 1
    return self.sampler.walk_logits(self.state, 1, [(self.rows[e['id']], 0) for e in entries for _ in e['want']])

  def step(self, entries, end):
    """Runs one step; logits f32 [wanted, vocab] on the host, or None when nothing is wanted."""
    known = [e['id'] in self.rows for e in entries]
    logits = None
    if entries:
      if all(known):
        logits = self._go_on(entries)
      elif not any(known):
        logits = self._start(entries)
      else:
        raise ValueError('a request joins a batch that has started')
      self.sampler.check_device_status(self.state)
    for i in end:
      self.rows.pop(i)
      self.lengths.pop(i)
    if not self.rows and self.state is not None:
      self.state = None
      self.sampler.delete_cache()
    if logits is None or not logits.shape[0]:
      return None
    return logits.cpu().numpy()


def main(argv=None):
  ap = argparse.ArgumentParser(prog='trace_run', description='Replay token ids through a model and write logits.')
  ap.add_argument('--model', required=True, help='folder with config.json and *.safetensors')
  ap.add_argument('--dtype', required=True, choices=['bfloat16', 'float32'])
  ap.add_argument('--out', required=True, help='folder for <step>.f32')
  ap.add_argument('--max-tokens', required=True, type=int, help='most tokens that live requests hold at any time')
  args = ap.parse_args(argv)
  from tunix_amd import build, registry
  if args.dtype not in registry.entry_of(registry.read_config(args.model)).dtypes:
    print(f'trace_run: this model does not run in {args.dtype}', file=sys.stderr)
    return 3
  build.ensure()
  replay = Replay(registry.load_model(args.model, args.dtype), args.max_tokens)
  for line in sys.stdin:
    if not line.strip():
      continue
    step = json.loads(line)
    logits = replay.step(step['entries'], step.get('end', []))
    if logits is not None:
      with open(os.path.join(args.out, f'{step["step"]}.f32'), 'wb') as f:
        f.write(np.ascontiguousarray(logits, dtype='<f4').tobytes())
    print(f'done {step["step"]}', flush=True)
  return 0


if __name__ == '__main__':
  sys.exit(main())
