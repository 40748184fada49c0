"""Latent-attention decoders without a GPU: configuration, weight layout, registry, trace replay bookkeeping, argument
checks of the C ABI, and the plain implementation's own checks (that a fault of a mechanism would show)."""
import copy
import ctypes
import json

import numpy as np
import pytest
import torch

import latent_common as LC
from oracle import latent as OL
from tunix_amd import _lib, latent, registry
from tunix_amd.latent import LatentConfig, LatentModel, Rotation, YarnScaling


def tokens(cfg, n, seed=1):
  return np.random.default_rng(seed).integers(0, cfg['vocab'], n)


# -- configuration -------------------------------------------------------------
def test_configuration_reads_every_size_and_constant():
  raw = LC.CONFIGS['mixed']
  c = LatentConfig.from_dict(raw)
  assert (c.vocab_size, c.embed_dim, c.streams, c.max_positions) == (101, 80, 2, 300)
  assert (c.norm_eps, c.logit_scale, c.num_layers) == (1e-5, 0.7, 4)
  l = c.layers[0]
  assert (l.heads, l.dim, l.rot_dim, l.vdim, l.kv_rank, l.ff, l.kv_from) == (3, 24, 16, 40, 72, 144, None)
  assert l.rot == Rotation(16, 5000.0, YarnScaling(4.0, 64.0, 4.0, 1.0)) and l.gate and not l.sink
  assert c.layers[1].ff is None and c.layers[1].sink and not c.layers[1].gate
  assert c.layers[2].kv_from == 1 and c.layers[3].rot.scaling is None


@pytest.mark.parametrize('edit, text', [
    (lambda c: c['layers'][0].update(type='other'), 'unknown mixer'),
    (lambda c: c['layers'][0]['mlp'].update(kind='sparse'), 'feed-forward kind'),
    (lambda c: c['layers'][2]['mixer'].update(kv_from=2), 'not an earlier layer'),
    (lambda c: c['layers'][3]['mixer'].update(kv_from=1), 'no latents of its own of the same sizes'),
    (lambda c: c['layers'][3]['mixer'].update(kv_from=2), 'no latents of its own'),
    (lambda c: c['layers'][0]['mixer'].update(kv_rank=600), 'up to 512'),
    (lambda c: c['layers'][0]['mixer']['rot'].update(dims=8), 'rotation covers'),
    (lambda c: c.update(streams=9), 'residual streams'),
])
def test_configurations_outside_what_the_kernels_do_are_refused(edit, text):
  raw = copy.deepcopy(LC.CONFIGS['mixed'])
  edit(raw)
  with pytest.raises(ValueError, match=text):
    LatentConfig.from_dict(raw)


@pytest.mark.parametrize('r', [LC.rot(16, 5000.0), LC.rot(2, 7.0), LC.rot(64, 1e6, LC.YARN),
                               LC.rot(32, 1e4, {'factor': 1.5, 'original': 512, 'fast': 32.0, 'slow': 1.0}),
                               LC.rot(8, 1e4, {'factor': 8.0, 'original': 8, 'fast': 64.0, 'slow': 32.0})])
def test_rotation_table_is_the_plain_rotation(r):
  s = r.get('scaling')
  product = Rotation(r['dims'], r['base'], YarnScaling(**s) if s else None)
  f, mult = OL.rotary_frequencies(r)
  pf, pm = product.frequencies()
  np.testing.assert_allclose(pf, f, rtol=1e-14)
  assert pm == mult and (mult == 1.0) == (s is None)
  t = product.table(50).numpy()
  x = np.random.default_rng(0).standard_normal((50, r['dims']))
  h = r['dims'] // 2
  u, v = x[:, :h], x[:, h:]
  got = np.concatenate([u * t[..., 0] - v * t[..., 1], v * t[..., 0] + u * t[..., 1]], -1)
  np.testing.assert_allclose(got, OL.rotate(x, np.arange(50), r), atol=1e-5)


# -- weights --------------------------------------------------------------------
def unpack(m):
  """DenseMatrix -> [heads, N, K] f32."""
  if m.w.dtype == torch.float32:
    return m.w.reshape(m.heads, m.n, m.k)
  v, d = m.heads * m.n, m.k
  t = m.w.reshape(v // 32, d // 64, 4, 2, 32, 8).permute(0, 4, 1, 3, 2, 5)
  return t.reshape(m.heads, m.n, m.k).float()


@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
@pytest.mark.parametrize('name', sorted(LC.CONFIGS))
def test_weights_sit_where_the_kernels_read_them_and_padding_is_zero(name, dtype):
  cfg = LC.CONFIGS[name]
  st = LC.make_state(cfg, 3)
  m = LC.product(cfg, st, dtype, device='cpu')
  d = cfg['width']
  for i, (l, w) in enumerate(zip(m.config.layers, m.layers)):
    off_qr, off_kv, off_gate, total = l.columns()
    z = unpack(w['in'])[0].numpy()
    assert z.shape[0] == total and total % 32 == 0
    want = np.zeros_like(z)
    q = st[f'l{i}.mix.q'].reshape(l.heads, l.dim + l.rot_dim, d)
    for h in range(l.heads):
      want[h * l.dim_p:h * l.dim_p + l.dim, :d] = q[h, :l.dim]
      want[off_qr + h * l.rot_dim:off_qr + (h + 1) * l.rot_dim, :d] = q[h, l.dim:]
      if l.gate:
        want[off_gate + h * l.vdim_p:off_gate + h * l.vdim_p + l.vdim, :d] = st[f'l{i}.mix.g'][h * l.vdim:(h + 1) * l.vdim]
    if l.kv_from is None:
      want[off_kv:off_kv + l.kv_rank + l.rot_dim, :d] = st[f'l{i}.mix.dkv']
    else:
      assert off_kv == -1
    np.testing.assert_array_equal(z, want)
    uk, uv = unpack(w['uk']).numpy(), unpack(w['uv']).numpy()
    o = unpack(w['o'])[0].numpy().reshape(-1, l.heads, l.vdim_p)
    for h in range(l.heads):
      np.testing.assert_array_equal(uk[h, :l.kv_rank, :l.dim], st[f'l{i}.mix.uk'][h * l.dim:(h + 1) * l.dim].T)
      np.testing.assert_array_equal(uv[h, :l.vdim, :l.kv_rank], st[f'l{i}.mix.uv'][h * l.vdim:(h + 1) * l.vdim])
      np.testing.assert_array_equal(o[:d, h, :l.vdim], st[f'l{i}.mix.o'][:, h * l.vdim:(h + 1) * l.vdim])
    assert not uk[:, l.kv_rank:].any() and not uk[:, :, l.dim:].any()
    assert not uv[:, l.vdim:].any() and not uv[:, :, l.kv_rank:].any() and not o[d:].any() and not o[:, :, l.vdim:].any()
    if l.ff is not None:
      gu = unpack(w['gate_up'])[0].numpy()
      fp = gu.shape[0] // 2
      np.testing.assert_array_equal(gu[:l.ff, :d], st[f'l{i}.mlp.gate'])
      np.testing.assert_array_equal(gu[fp:fp + l.ff, :d], st[f'l{i}.mlp.up'])
      np.testing.assert_array_equal(w['gate_up'].bias.numpy()[fp:fp + l.ff], st[f'l{i}.mlp.up.b'])
      assert not gu[l.ff:fp].any() and not w['gate_up'].bias.numpy()[l.ff:fp].any()
      np.testing.assert_array_equal(unpack(w['down'])[0].numpy()[:d, :l.ff], st[f'l{i}.mlp.down'])


def test_state_must_fit_the_configuration():
  cfg = LC.CONFIGS['one']
  st = {k: torch.from_numpy(v) for k, v in LC.make_state(cfg).items()}
  c = LatentConfig.from_dict(cfg)
  with pytest.raises(KeyError, match='missing'):
    LatentModel.from_state(c, {k: v for k, v in st.items() if k != 'l0.mix.sink'}, device='cpu')
  with pytest.raises(KeyError, match='unexpected'):
    LatentModel.from_state(c, {**st, 'l0.mix.extra': st['pos']}, device='cpu')
  with pytest.raises(ValueError, match='shape'):
    LatentModel.from_state(c, {**st, 'pos': st['pos'][:3]}, device='cpu')


def test_cache_views_tile_the_cache():
  c = LatentConfig.from_dict(LC.CONFIGS['mixed'])
  b, size = 3, 40
  cache = torch.zeros(c.cache_shape(b, size))
  views = c.cache_rows(cache, b, size)
  assert len(views) == 3                              # the third layer reads the second one's latents
  assert [v.shape[-1] for v in views] == [128 + 64, 64 + 64, 128 + 64]
  for v in views:
    v += 1
  assert bool((cache == 1).all())


# -- registry ---------------------------------------------------------------------
def save_model(folder, cfg, state):
  from safetensors.torch import save_file
  folder.mkdir(exist_ok=True)
  (folder / 'config.json').write_text(json.dumps(cfg))
  save_file({k: torch.from_numpy(v).to(torch.bfloat16) for k, v in state.items()}, str(folder / 'model.safetensors'))


def test_registry_builds_the_model_config_json_names(tmp_path):
  cfg = LC.CONFIGS['mixed']
  save_model(tmp_path / 'm', cfg, LC.make_state(cfg))
  m = registry.load_model(str(tmp_path / 'm'), 'float32', device='cpu')
  assert isinstance(m, LatentModel) and m.dtype == torch.float32 and m.config == LatentConfig.from_dict(cfg, 'float32')
  hf = {'architectures': ['Qwen3ForCausalLM'], 'num_hidden_layers': 2, 'vocab_size': 128, 'hidden_size': 64,
        'intermediate_size': 128, 'num_attention_heads': 4, 'num_key_value_heads': 2, 'head_dim': 16, 'rms_norm_eps': 1e-6,
        'rope_theta': 5e5, 'tie_word_embeddings': True}
  (tmp_path / 'q').mkdir()
  (tmp_path / 'q' / 'config.json').write_text(json.dumps(hf))
  c = registry.load_config(str(tmp_path / 'q'))
  assert (c.family, c.num_layers, c.head_dim, c.num_kv_heads, c.rope_theta, c.weight_tying) == ('qwen3', 2, 16, 2, 5e5, True)
  with pytest.raises(ValueError, match='not in float32'):
    registry.load_config(str(tmp_path / 'q'), 'float32')
  (tmp_path / 'q' / 'config.json').write_text(json.dumps({'architecture': 'Nothing'}))
  with pytest.raises(ValueError, match='unknown architecture'):
    registry.load_config(str(tmp_path / 'q'))


def test_trace_run_refuses_a_format_the_model_does_not_have(tmp_path):
  from tunix_amd import trace
  (tmp_path / 'config.json').write_text(json.dumps({'architectures': ['LlamaForCausalLM']}))
  assert trace.main(['--model', str(tmp_path), '--dtype', 'float32', '--out', str(tmp_path), '--max-tokens', '8']) == 3


# -- trace replay -------------------------------------------------------------------
class _Recorder:
  """Stands for the device: remembers what each walk was asked for and returns numbered logits."""

  def __init__(self, monkeypatch, vocab):
    from tunix_amd.sampler import Sampler
    self.calls = []
    rec = self

    def walk(sampler, st, n, wanted):
      rec.calls.append((st['token_buffer'].clone(), n, list(wanted), sampler.cache_config.cache_size))
      return torch.arange(len(wanted) * vocab, dtype=torch.float32).reshape(len(wanted), vocab)

    monkeypatch.setattr(Sampler, 'walk_logits', walk)
    monkeypatch.setattr(Sampler, 'check_device_status', lambda s, st: None)


def test_replay_pads_on_the_left_and_keeps_rows_of_a_batch(monkeypatch):
  from tunix_amd.trace import Replay
  cfg = LC.CONFIGS['one']
  m = LC.product(cfg, LC.make_state(cfg), device='cpu')
  rec = _Recorder(monkeypatch, 64)
  r = Replay(m, 30)
  e = lambda i, t, w=(): {'id': i, 'tokens': list(t), 'want': list(w)}
  out = r.step([e('a', [5, 6, 7], [0, 2]), e('b', [9])], [])
  buf, n, wanted, size = rec.calls[-1]
  assert n == 3 and buf[0, :3].tolist() == [5, 6, 7] and buf[1, :3].tolist() == [0, 0, 9]
  assert wanted == [(0, 0), (0, 2)] and out.shape == (2, 64)
  assert r.state['input_mask_host'][1, :4].tolist() == [False, False, True, True]
  assert r.state['positions_host'][1, 2:5].tolist() == [0, 1, 2] and size >= 3 + 29
  assert r.step([e('b', [11], [0]), e('a', [10])], ['a']).shape == (1, 64)        # entries in another order
  buf, n, wanted, _ = rec.calls[-1]
  assert n == 1 and buf[:, 3].tolist() == [10, 11] and wanted == [(1, 0)]
  assert r.step([e('b', [12])], ['b']) is None                                    # nothing wanted, row a has ended
  assert rec.calls[-1][0][:, 4].tolist() == [0, 12] and r.state is None and r.sampler._cache is None
  r.step([e('c', [1, 2])], [])
  with pytest.raises(ValueError, match='joins'):
    r.step([e('c', [1]), e('d', [1])], [])
  with pytest.raises(ValueError, match='batch before them has ended'):
    r.step([e('d', [1])], [])
  with pytest.raises(ValueError, match='vocabulary'):
    r.step([e('c', [64])], [])


def test_sequences_beyond_the_position_table_are_rejected():
  import common as C
  from tunix_amd.configs import CacheConfig
  from tunix_amd.sampler import Sampler
  cfg = LC.config(LC.CONFIGS['one']['layers'], vocab=64, width=36, streams=1, max_positions=8)
  m = LC.product(cfg, LC.make_state(cfg), device='cpu')
  s = Sampler(m, C.ToyTokenizer(), CacheConfig(64, m.config.num_layers, m.config.num_kv_heads, m.config.head_dim))
  with pytest.raises(ValueError, match='exceeds the 8 positions'):
    s(prompt_token_ids=[[3, 4, 5, 6, 7]], max_generation_steps=4)
  assert s.transformer_state == {}
  with pytest.raises(ValueError, match='same structure'):
    s.update_params({'layers.0.attn.q_proj.w_lora_a': np.zeros((2, 2), np.float32)})


# -- C ABI without a device ------------------------------------------------------------
def test_argument_checks_of_the_latent_entry_points():
  lib = _lib.lib()
  p = 0x1000
  assert lib.tmx_dense_linear(None, 0, None, 64, 0, p, None, None, 0, p, 64, 0, 1, 64, 64, 1, 0) == -1
  assert lib.tmx_dense_linear(None, 0, p, 64, 0, p, None, None, 0, p, 64, 0, 1, 65, 64, 1, 0) == -2
  assert lib.tmx_dense_linear(None, 0, p, 64, 0, p, None, None, 0, p, 64, 0, 1, 64, 64, 1, 2) == -1   # no gate
  assert lib.tmx_dense_linear(None, 0, p, 64, 0, p, None, None, 0, p, 64, 0, 1, 64, 64, 1, 9) == -4
  assert lib.tmx_dense_linear(None, 0, p, 64, 0, p, p, None, 0, p, 64, 0, 1, 64, 64, 2, 0) == -1      # bias and heads
  assert lib.tmx_stream_rows(None, 0, p, None, None, None, p, p, p, 4, 9, 64, 64, 1e-5, 1) == -2
  assert lib.tmx_stream_rows(None, 0, p, p, None, p, p, p, p, 4, 2, 64, 64, 1e-5, 1) == -1
  assert lib.tmx_latent_attention(None, 0, p, p, None, p, p, 8, p, None, 1, 1, 4, 96, 64, 8, 1.0) == -2
  assert lib.tmx_latent_rows(None, 0, p, 64, 0, 0, None, 1e-5, p, 8, p, p, 8, p, p, 1, 1, 1, 4, 8, 64, 64, 8) == -1
  assert lib.tmx_latent_attention_workspace_bytes(300, 1, 8, 64, 64) == 0
  assert lib.tmx_latent_attention_workspace_bytes(1, 1, 8, 64, 1024) > 0


@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
def test_step_descriptor_is_accepted_and_its_faults_are_not(dtype):
  lib = _lib.lib()
  m = LC.product(LC.CONFIGS['mixed'], LC.make_state(LC.CONFIGS['mixed']), dtype, device='cpu')
  d = m.desc()
  n = lib.tmx_decode_workspace_bytes(ctypes.byref(d), 4, 64)
  assert 0 < n < lib.tmx_decode_workspace_bytes(ctypes.byref(d), 400, 64)
  for field, bad in (('streams', 9), ('act', 7), ('max_positions', 0)):
    good = getattr(d, field)
    setattr(d, field, bad)
    assert lib.tmx_decode_workspace_bytes(ctypes.byref(d), 4, 64) == 0
    setattr(d, field, good)
  a = m._keep[2]
  for field, bad in (('kv_layer', 2), ('kv_layer', 0), ('rank_p', 96), ('heads', 0), ('off_qr', 0)):
    good = getattr(a, field)
    setattr(a, field, bad)
    assert lib.tmx_decode_workspace_bytes(ctypes.byref(d), 4, 64) == 0, field
    setattr(a, field, good)
  assert lib.tmx_decode_workspace_bytes(ctypes.byref(d), 4, 64) == n


# -- the plain implementation -----------------------------------------------------------
def _faults():
  """name -> (configuration, state) -> the same with one mechanism left out or changed."""
  def cfg_edit(fn):
    def go(cfg, st):
      cfg = copy.deepcopy(cfg)
      fn(cfg)
      return cfg, st
    return go

  def st_edit(fn):
    def go(cfg, st):
      st = dict(st)
      fn(st)
      return cfg, st
    return go

  return {
      'no sink': st_edit(lambda s: s.update({'l1.mix.sink': np.full_like(s['l1.mix.sink'], -1e4)})),
      'no gate': st_edit(lambda s: s.update({'l0.mix.g': np.zeros_like(s['l0.mix.g'])})),
      'no yarn': cfg_edit(lambda c: c['layers'][0]['mixer']['rot'].pop('scaling')),
      'other base': cfg_edit(lambda c: c['layers'][3]['mixer']['rot'].update(base=9000.0)),
      'other scale': cfg_edit(lambda c: c['layers'][1]['mixer'].update(scale=c['layers'][1]['mixer']['scale'] * 1.05)),
      'no position vector': st_edit(lambda s: s.update({'pos': np.zeros_like(s['pos'])})),
      'mix transposed': st_edit(lambda s: s.update({'l0.hc1.mix': s['l0.hc1.mix'].T.copy()})),
      'no bias': st_edit(lambda s: s.update({'l3.mlp.down.b': np.zeros_like(s['l3.mlp.down.b'])})),
      'other eps': cfg_edit(lambda c: c['norm'].update(eps=1e-2)),
      'other logit scale': cfg_edit(lambda c: c.update(logit_scale=0.75)),
  }


@pytest.mark.parametrize('fault', sorted(_faults()))
def test_a_fault_of_one_mechanism_shows_in_the_logits(fault):
  """The tolerances of the device tests are far below what leaving a mechanism out changes."""
  cfg = LC.CONFIGS['mixed']
  st = LC.make_state(cfg, 5)
  t = tokens(cfg, 40)
  want = LC.plain(cfg, st, t)
  bad_cfg, bad_st = _faults()[fault](cfg, st)
  assert LC.error(LC.plain(bad_cfg, bad_st, t), want) > 3 * LC.LIMIT['float32'] * 10
  if fault not in ('other eps', 'other scale', 'other base'):
    assert LC.error(LC.plain(bad_cfg, bad_st, t), want) > 1.5 * LC.LIMIT['bfloat16']


def test_the_roundings_of_the_bf16_form_stay_within_its_tolerance():
  for name, cfg in LC.CONFIGS.items():
    st = LC.make_state(cfg, 6)
    t = tokens(cfg, 33)
    assert 0 < LC.error(LC.plain(cfg, st, t, 'bfloat16'), LC.plain(cfg, st, t)) < LC.LIMIT['bfloat16'], name


def test_plain_attention_is_causal():
  cfg = LC.CONFIGS['mixed']
  st = LC.make_state(cfg, 7)
  t = tokens(cfg, 30)
  other = t.copy()
  other[20:] = (other[20:] + 1) % cfg['vocab']
  a, b = LC.plain(cfg, st, t), LC.plain(cfg, st, other)
  np.testing.assert_array_equal(a[:20], b[:20])
  assert np.abs(a[20:] - b[20:]).max() > 0.1
