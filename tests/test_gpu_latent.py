"""Latent-attention decoders on the GPU: every mechanism alone against the plain implementation's function, then whole
models (both number formats) through the Sampler: prompts, decoding, portions, mixed batches, reused caches, long
sequences, generation and the trace command."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import common as C
import gpu_util as G
import latent_common as LC
from gpu_util import act, all_logits, dev, rounded, sampler, up
from oracle import latent as OL
from oracle.bf16 import bf16_round
from tunix_amd import _lib
from tunix_amd.configs import RolloutConfig
from tunix_amd.latent import pack_tiles

pytestmark = pytest.mark.gpu
S = _lib.stream
FORMATS = ['float32', 'bfloat16']


# -- mechanisms alone -------------------------------------------------------------
@pytest.mark.parametrize('dtype', FORMATS)
@pytest.mark.parametrize('epi', [0, 1, 2, 3])
def test_dense_projection(dtype, epi):
  """Row counts on both sides of every kernel form's limits, K from one tile up, several matrices side by side."""
  rng = np.random.default_rng(epi)
  for m, k, n, heads in [(1, 64, 64, 1), (5, 128, 192, 1), (33, 320, 64, 1), (64, 1024, 128, 1), (100, 64, 256, 1),
                         (128, 576, 64, 1), (130, 192, 320, 1), (257, 256, 448, 1), (300, 64, 64, 1), (515, 1088, 128, 1),
                         (3, 64, 96, 3), (40, 256, 64, 5), (200, 128, 32, 4), (700, 512, 128, 2)]:
    if epi == 1 and (heads > 1 or n % 64):
      continue
    print('dense', dtype, epi, m, k, n, heads, flush=True)
    x = rounded(rng.standard_normal((m, heads, k)).astype(np.float32), dtype)
    w = rounded((rng.standard_normal((heads, n, k)) * k ** -0.5).astype(np.float32), dtype)
    bias = rng.standard_normal(n).astype(np.float32) if heads == 1 else None
    gate = rounded(rng.standard_normal((m, heads, n)).astype(np.float32), dtype)
    y = np.einsum('mhk,hnk->mhn', x.astype(np.float64), w)
    if bias is not None:
      y = y + bias
    if epi == 1:
      g, u = y[..., :n // 2], y[..., n // 2:]
      y = g * OL.sigmoid(g) * u
    elif epi == 2:
      y = y * OL.sigmoid(gate.astype(np.float64))
    elif epi == 3:
      y = np.maximum(y, 0.0) ** 2
    wt = torch.from_numpy(w.reshape(heads * n, k))
    wt = wt.to(G.DEV) if dtype == 'float32' else pack_tiles(wt.to(torch.bfloat16)).to(G.DEV)
    keep = [dev(x, dtype), wt, None if bias is None else G.f32(bias), dev(gate, dtype)]
    out = dev(np.full((m, heads, y.shape[-1]), np.nan, np.float32), dtype)
    G.call('tmx_dense_linear', S(), act(dtype), G.p(keep[0]), heads * k, k, G.p(wt), G.p(keep[2]), G.p(keep[3]),
           heads * n, G.p(out), heads * y.shape[-1], y.shape[-1], m, k, n, heads, epi)
    G.sync()
    got = G.host(out)
    tol = 3e-6 if dtype == 'float32' else 6e-3
    assert np.abs(got - y).max() <= tol * max(1.0, np.abs(y).max()), (m, k, n, heads)


@pytest.mark.parametrize('dtype', FORMATS)
@pytest.mark.parametrize('streams', [1, 2, 3, 5, 8])
def test_stream_rows(dtype, streams):
  rng = np.random.default_rng(streams)
  for m, d in [(3, 36), (65, 192), (7, 2304)]:
    dp = up(d, 64)
    pad = lambda a: np.pad(a, [(0, 0)] * (a.ndim - 1) + [(0, dp - d)])
    xs = pad(rng.standard_normal((m, streams, d)).astype(np.float32))
    y = pad(rounded(rng.standard_normal((m, d)).astype(np.float32), dtype))
    mix, out, inn = (rng.standard_normal(s).astype(np.float32) for s in ((streams, streams), streams, streams))
    nw = pad(rng.standard_normal(d).astype(np.float32))
    eps = 0.02
    for update in (True, False):
      for store in (1, 0):
        hc = {'mix': mix, 'out': out}
        new = OL.mix_streams(xs.transpose(1, 0, 2).astype(np.float64), hc, y) if update else xs.transpose(1, 0, 2)
        u = np.einsum('s,snd->nd', inn, new)
        want = OL.rms_norm(u[:, :d], nw[:d], eps)
        x, yt = G.f32(xs), dev(y, dtype) if update else None
        xn = dev(np.full((m, dp), np.nan, np.float32), dtype)
        k = [G.f32(mix), G.f32(out), G.f32(inn), G.f32(nw)]
        G.call('tmx_stream_rows', S(), act(dtype), G.p(x), G.p(yt), *(G.p(t) for t in k), G.p(xn), m, streams, d, dp, eps, store)
        G.sync()
        got = G.host(xn)
        assert not got[:, d:].any()
        np.testing.assert_allclose(got[:, :d], want, atol=2e-6 if dtype == 'float32' else 2e-2, rtol=1e-5 if dtype == 'float32' else 8e-3)
        np.testing.assert_allclose(G.host(x), new.transpose(1, 0, 2) if (store and update) else xs, atol=1e-5, rtol=1e-5)


@pytest.mark.parametrize('dtype', FORMATS)
@pytest.mark.parametrize('own', [True, False])
def test_latent_rows(dtype, own):
  """Rotation at the row's position, norm of the latent, zero padding; one and several tokens per pass; positions that
  start late (padding on the left) and one past the table (clamped)."""
  from tunix_amd.latent import Rotation, YarnScaling
  rng = np.random.default_rng(7)
  for H, rot, rank, T, nseq in [(3, 4, 12, 1, 5), (2, 66, 300, 3, 2), (7, 32, 64, 5, 3)]:
    rank_p, rot_p = next(p for p in (64, 128, 256, 512) if rank <= p), 64 if rot <= 64 else 128
    ld, cs, buf, maxpos, step, eps = rank_p + rot_p, 40, 50, 30, 6, 1e-3
    r = LC.rot(rot, 500.0, LC.YARN)
    table = Rotation(rot, 500.0, YarnScaling(**LC.YARN)).table(maxpos).to(G.DEV)
    m = nseq * T
    off_qr, off_kv = 64, up(64 + H * rot, 32)
    ldz = off_kv + up(rank + rot, 32)
    z = rounded(rng.standard_normal((m, ldz)).astype(np.float32), dtype)
    nw = rng.standard_normal(rank).astype(np.float32)
    first = rng.integers(0, 5, nseq)
    pos = np.maximum(np.arange(buf)[None] - first[:, None], 0).astype(np.int32)
    pos[-1] += maxpos - step - 2     # the last rows' positions run over the end of the table
    zt, qt = dev(z, dtype), dev(np.full((m, H, ld), 7.0, np.float32), dtype)
    cache = dev(np.zeros((nseq, cs, ld), np.float32), dtype)
    k = [G.f32(nw), G.i32(pos), G.i32([step])]
    G.call('tmx_latent_rows', S(), act(dtype), G.p(zt), ldz, off_qr, off_kv if own else -1, G.p(k[0]), eps,
           table.data_ptr(), maxpos, G.p(k[1]), G.p(k[2]), buf, G.p(qt), G.p(cache), m, T, H, rot, rank, rank_p, rot_p, cs)
    G.sync()
    q, ch = G.host(qt), G.host(cache)
    tol = dict(atol=3e-6, rtol=1e-5) if dtype == 'float32' else dict(atol=2e-2, rtol=8e-3)
    assert (q[:, :, :rank_p] == 7.0).all() and not q[:, :, rank_p + rot:].any()
    for i in range(m):
      slot = step + i % T
      p = np.array([min(pos[i // T, slot], maxpos - 1)])
      want = OL.rotate(z[i, off_qr:off_qr + H * rot].reshape(H, 1, rot).astype(np.float64), p, r)[:, 0]
      np.testing.assert_allclose(q[i, :, rank_p:rank_p + rot], want, **tol)
      row = ch[i // T, slot]
      if not own:
        assert not row.any()
        continue
      np.testing.assert_allclose(row[:rank], OL.rms_norm(z[i, off_kv:off_kv + rank].astype(np.float64), nw, eps), **tol)
      np.testing.assert_allclose(row[rank_p:rank_p + rot],
                                 OL.rotate(z[i:i + 1, off_kv + rank:off_kv + rank + rot].astype(np.float64), p, r)[0], **tol)
      assert not row[rank:rank_p].any() and not row[rank_p + rot:].any()
    written = np.zeros((nseq, cs), bool)
    written[:, step:step + T] = own
    assert not ch[~written].any()


def attention_case(dtype, rank_p, rot_p, H, T, nseq, step, cs, sink, seed, far=None, mask_first=0):
  """Runs tmx_latent_attention and returns (got, want) [m, H, rank_p]; far: (query row, slot) whose score stands out."""
  rng = np.random.default_rng(seed)
  ld, m, buf = rank_p + rot_p, nseq * T, cs + 3
  q = rng.standard_normal((m, H, ld)).astype(np.float32)
  cache = rng.standard_normal((nseq, cs, ld)).astype(np.float32)
  if far:
    row, slot = far
    q[row] *= 0.3
    cache[row // T, slot] = np.sign(q[row, 0]) * 2.5     # one score about 10 above the rest
  q, cache = rounded(q, dtype), rounded(cache, dtype)
  scale = ld ** -0.5
  mask = np.ones((nseq, buf), np.uint8)
  for s in range(nseq):
    mask[s, :min(mask_first * s, step)] = 0
  snk = (2.0 * rng.standard_normal(H)).astype(np.float32) if sink else None
  want = np.zeros((m, H, rank_p))
  for i in range(m):
    s, lim = i // T, step + i % T
    ok = np.flatnonzero(mask[s, :lim + 1])
    sc = (q[i].astype(np.float64) @ cache[s, ok].T.astype(np.float64)) * scale
    top = np.maximum(sc.max(-1), snk) if sink else sc.max(-1)
    e = np.exp(sc - top[:, None])
    den = e.sum(-1) + (np.exp(snk - top) if sink else 0)
    want[i] = e @ cache[s, ok, :rank_p].astype(np.float64) / den[:, None]
  # slots behind the newest one hold large garbage, the rows past every limit too
  junk = cache.copy()
  junk[:, step + T:] = 50.0
  out = dev(np.full((m, H, rank_p), np.nan, np.float32), dtype)
  nb = _lib.lib().tmx_latent_attention_workspace_bytes(nseq, T, H, rank_p, cs)
  ws = torch.empty(max(nb, 4), dtype=torch.uint8, device=G.DEV)
  k = [dev(q, dtype), dev(junk, dtype), None if snk is None else G.f32(snk), G.u8(mask), G.i32([step])]
  G.call('tmx_latent_attention', S(), act(dtype), *(G.p(t) for t in k), buf, G.p(out), G.p(ws), nseq, T, H, rank_p, rot_p,
         cs, scale)
  G.sync()
  return G.host(out), want


@pytest.mark.parametrize('dtype', FORMATS)
@pytest.mark.parametrize('rank_p, rot_p', [(64, 64), (128, 128), (256, 64), (256, 128), (512, 64), (512, 128)])
def test_latent_attention(dtype, rank_p, rot_p):
  """One and many tokens per pass, few and many heads (both forms of the walk), every remainder of a block of 32
  positions, one and several splits, padding on the left, with and without a sink."""
  seed = 0
  for H, T, nseq, step, cs in [(1, 1, 2, 0, 40), (6, 1, 3, 31, 64), (16, 1, 1, 700, 800), (32, 1, 2, 64, 70), (33, 1, 2, 95, 96),
                               (5, 2, 2, 30, 64), (40, 4, 1, 100, 300), (3, 37, 2, 5, 60), (9, 128, 1, 0, 128), (8, 1, 300, 40, 64)]:
    for sink in (False, True):
      seed += 1
      print('latent attention', dtype, rank_p, rot_p, H, T, nseq, step, cs, sink, flush=True)
      got, want = attention_case(dtype, rank_p, rot_p, H, T, nseq, step, cs, sink, seed, mask_first=3)
      tol = 2e-5 if dtype == 'float32' else 1.2e-2
      assert np.abs(got - want).max() <= tol * max(1.0, np.abs(want).max()), (H, T, nseq, step, cs, sink)


@pytest.mark.parametrize('dtype', FORMATS)
def test_a_single_far_key_decides_the_output(dtype):
  """A key whose score stands out, at both ends of blocks of 32 slots and of the visible range: just visible ones decide
  the output, one slot further they do not exist."""
  for T, step in ((1, 300), (16, 284)):
    for slot in (0, 1, 31, 32, 63, 64, 255, 256, 298, 299, 300):
      row = min(max(slot - step, 0), T - 1)
      got, want = attention_case(dtype, 128, 64, 4, T, 1, step, 320, True, slot, far=(row, slot))
      assert np.abs(got - want).max() <= (3e-5 if dtype == 'float32' else 3e-2) * np.abs(want).max(), (T, slot)
      strong = float(np.abs(want[row, 0]).mean()) > 1.2         # the key's value (2.5 in magnitude) is there ...
      assert strong == (slot <= step + T - 1), (T, slot)       # (slot 300 lies behind the last of 16 tokens at 284)
      if T > 1 and 0 < slot - step < T:                        # ... and not for the token before it
        assert float(np.abs(want[row - 1, 0]).mean()) < 1.0


# -- whole models -------------------------------------------------------------------
_built = {}


def model(name, dtype, seed=11):
  if (name, dtype, seed) not in _built:
    st = LC.make_state(LC.CONFIGS[name], seed)
    _built[name, dtype, seed] = LC.product(LC.CONFIGS[name], st, dtype), st
  return _built[name, dtype, seed]


_plain = {}


def plain(name, st, t, dtype):
  key = (name, dtype, tuple(int(x) for x in t))
  if key not in _plain:
    _plain[key] = LC.plain(LC.CONFIGS[name], st, t, dtype)
  return _plain[key]


def toks(name, n, seed):
  return np.random.default_rng(seed).integers(0, LC.CONFIGS[name]['vocab'], n)


@pytest.mark.parametrize('dtype', FORMATS)
@pytest.mark.parametrize('name', sorted(LC.CONFIGS))
def test_prompt_logits(name, dtype):
  m, st = model(name, dtype)
  for n in (1, 2, 33, 200):
    t = toks(name, n, n)
    got = all_logits(sampler(m, 256), [t], 256)[0]
    assert LC.error(got, plain(name, st, t, dtype)) < LC.LIMIT[dtype], n


@pytest.mark.parametrize('dtype', FORMATS)
@pytest.mark.parametrize('name', sorted(LC.CONFIGS))
def test_portions_and_token_by_token_decoding(name, dtype):
  """However the tokens are cut, down to two and one at a time, the logits are those of the whole prompt."""
  m, st = model(name, dtype)
  t = toks(name, 97, 5)
  want = plain(name, st, t, dtype)
  for cuts in ([1] * 97, [2] * 48 + [1], [3] * 32 + [1], [64, 33], [31, 1, 1, 32, 32], [96, 1], [7] * 13 + [6]):
    got = all_logits(sampler(m, 128), [t], 128, cuts)[0]
    assert LC.error(got, want) < LC.LIMIT[dtype], cuts[:4]


@pytest.mark.parametrize('dtype', FORMATS)
@pytest.mark.parametrize('name', sorted(LC.CONFIGS))
def test_unequal_requests_in_one_batch(name, dtype):
  """Rows of different lengths (padding on the left), each as if it were alone; more rows than one kernel form takes."""
  m, st = model(name, dtype)
  for lens in ((1, 50, 23, 2), (70, 69, 1), tuple(range(1, 41))):
    rows = [toks(name, n, 100 + n) for n in lens]
    got = all_logits(sampler(m, 128), rows, 128, [max(lens) - 3, 1, 2] if max(lens) > 40 else None)
    for r, g in zip(rows, got):
      assert LC.error(g, plain(name, st, r, dtype)) < LC.LIMIT[dtype], len(r)


@pytest.mark.parametrize('dtype', FORMATS)
def test_a_cache_that_is_used_again(dtype):
  """Batches of other shapes on one sampler, the cache kept or given back in between."""
  m, st = model('mixed', dtype)
  s = sampler(m, 128)
  for i, lens in enumerate([(90, 40), (3, 60), (90, 1), (5,), (2, 2, 2), (100,)]):
    rows = [toks('mixed', n, 200 + 10 * i + n) for n in lens]
    for r, g in zip(rows, all_logits(s, rows, 128, [max(lens) - 1, 1] if max(lens) > 3 else None)):
      assert LC.error(g, plain('mixed', st, r, dtype)) < LC.LIMIT[dtype], lens
    if i % 2:
      s.delete_cache()


@pytest.mark.parametrize('dtype', FORMATS)
def test_long_decoding(dtype):
  m, st = model('one', dtype)
  t = toks('one', 290, 9)
  got = all_logits(sampler(m, 300), [t], 300, [4] + [1] * 286)[0]
  want = plain('one', st, t, dtype)
  assert LC.error(got, want) < LC.LIMIT[dtype]
  assert LC.error(got[:4], want[:4]) < LC.LIMIT[dtype] and LC.error(got[-20:], want[-20:]) < LC.LIMIT[dtype]


@pytest.mark.parametrize('dtype', FORMATS)
def test_a_far_token_changes_later_logits_as_the_plain_model_says(dtype):
  """The first and a middle token replaced: the logits hundreds of tokens later move, and move as expected."""
  m, st = model('wide', dtype)
  st = dict(st)
  t = toks('wide', 260, 3)
  s = sampler(m, 300)
  base, want = all_logits(s, [t], 300)[0], plain('wide', st, t, dtype)
  for at in (0, 31, 32, 128):
    o = t.copy()
    o[at] = (o[at] + 5) % LC.CONFIGS['wide']['vocab']
    got, w2 = all_logits(s, [o], 300, [255] + [1] * 5)[0], plain('wide', st, o, dtype)
    assert LC.error(got, w2) < LC.LIMIT[dtype]
    move, expected = got[-1] - base[-1], w2[-1] - want[-1]
    assert np.abs(expected).max() > 0 and (dtype == 'bfloat16' or np.abs(move - expected).max() < 0.05 * np.abs(expected).max())


def test_more_rows_than_the_streaming_kernels_take():
  """Passes of more than 128 rows (the 256-row blocks, planes of split projections) and the head in both forms."""
  cfg = LC.config([LC.layer('latent_attention', 4, 48, 16, 64, 100, 1100), LC.layer('latent_attention_2', 4, 48, 16, 64, 100, 1100, kv_from=None)],
                  vocab=300, width=1088, streams=2, max_positions=64)
  st = LC.make_state(cfg, 2)
  rows = [np.random.default_rng(i).integers(0, 300, 40) for i in range(20)]
  want = [LC.plain(cfg, st, r, 'bfloat16') for r in rows[:3]]
  m = LC.product(cfg, st, 'bfloat16')
  for n in (3, 20):
    got = all_logits(sampler(m, 64), rows[:n], 64, [38, 1, 1])
    for g, w in zip(got, want):
      assert LC.error(g, w) < LC.LIMIT['bfloat16']
  # scoring passes take the wide head (width a multiple of 128): compare its log-probs with the logits'
  cfg = dict(cfg, width=1152)
  st = LC.make_state(cfg, 2)
  m = LC.product(cfg, st, 'bfloat16')
  s = sampler(m, 64)
  lp = s.per_token_logps(np.stack([r[:10] for r in rows]), np.stack([r[10:] for r in rows]), pad_id=0, token_mask=np.ones((20, 40), bool))
  z = LC.plain(cfg, st, rows[0])
  z = z - np.log(np.exp(z - z.max(-1, keepdims=True)).sum(-1, keepdims=True)) - z.max(-1, keepdims=True)
  ref = np.array([z[c - 1, rows[0][c]] for c in range(10, 40)])
  assert np.abs(lp[0] - ref).max() < 0.1


@pytest.mark.parametrize('dtype', FORMATS)
def test_projections_whose_k_is_split(dtype):
  """Long K in front of the streams: the slices' planes are added by the stream row kernel, in both kernel forms."""
  cfg = LC.config([LC.layer('latent_attention', 32, 20, 8, 60, 50, 4050), LC.layer('latent_attention_2', 17, 20, 8, 130, 50, 2100, kv_from=None)],
                  vocab=96, width=250, streams=3, max_positions=80)
  st = LC.make_state(cfg, 4)
  m = LC.product(cfg, st, dtype)
  rows = [np.random.default_rng(i).integers(0, 96, 24) for i in range(12)]
  want = [LC.plain(cfg, st, r, dtype) for r in rows[:2]]
  for n, cuts in ((1, [20, 1, 1, 2]), (2, [24]), (12, [22, 1, 1]), (12, [24])):
    got = all_logits(sampler(m, 32), rows[:n], 32, cuts)
    for g, w in zip(got, want):
      assert LC.error(g, w) < LC.LIMIT[dtype], (n, cuts)


# -- generation through the framework's entry points ------------------------------------
@pytest.mark.parametrize('dtype', FORMATS)
@pytest.mark.parametrize('name', ['mixed', 'wide'])
def test_greedy_generation(name, dtype):
  m, st = model(name, dtype)
  s = sampler(m, 96)
  prompts = [toks(name, n, 300 + n) for n in (5, 31, 12)]
  out = s(prompt_token_ids=prompts, max_generation_steps=24, eos_tokens=[-1], return_logprobs=True)
  checked = 0
  for p, got, lps in zip(prompts, out.tokens, out.logprobs):
    seq = np.concatenate([p, got])
    lg = plain(name, st, seq, 'float32')[len(p) - 1:-1]
    lp = lg - lg.max(-1, keepdims=True)
    lp -= np.log(np.exp(lp).sum(-1, keepdims=True))
    top = np.sort(lg, axis=-1)
    for i, (t, l) in enumerate(zip(got, lps)):
      slack = 1e-3 if dtype == 'float32' else 0.15
      assert lg[i].max() - lg[i, t] <= slack and abs(lp[i, t] - l) <= slack
      checked += top[i, -1] - top[i, -2] > slack and t == lg[i].argmax()
  assert checked > 30
  assert max(int(t.max()) for t in out.tokens) < LC.CONFIGS[name]['vocab']


@pytest.mark.parametrize('dtype', FORMATS)
def test_sampling_modes_logits_and_forbidden_ids(dtype):
  m, st = model('mixed', dtype)       # 101 ids: the head's padding rows must never be drawn
  s = sampler(m, 64)
  prompts = [toks('mixed', 9, i) for i in range(6)]
  for kw in (dict(temperature=3.0, top_p=1.0), dict(temperature=3.0, top_p=0.9), dict(temperature=5.0, top_p=1.0, top_k=40)):
    a = s(prompt_token_ids=prompts, max_generation_steps=16, eos_tokens=[-1], seed=3, return_logprobs=True, **kw)
    b = s(prompt_token_ids=prompts, max_generation_steps=16, eos_tokens=[-1], seed=3, return_logprobs=True, **kw)
    c = s(prompt_token_ids=prompts, max_generation_steps=16, eos_tokens=[-1], seed=4, return_logprobs=True, **kw)
    assert all((x == y).all() for x, y in zip(a.tokens, b.tokens)) and any((x != y).any() for x, y in zip(a.tokens, c.tokens))
    assert all(0 <= int(t) < 101 for r in a.tokens for t in r)
    z = plain('mixed', st, np.concatenate([prompts[0], a.tokens[0]]), 'float32')[8:-1] / kw['temperature']
    lp = z - z.max(-1, keepdims=True)
    lp -= np.log(np.exp(lp).sum(-1, keepdims=True))
    # (the sorting branch works on logits rounded to bf16 in both formats)
    exact = dtype == 'float32' and kw['top_p'] == 1.0 and 'top_k' not in kw
    np.testing.assert_allclose(a.logprobs[0], lp[np.arange(16), a.tokens[0]], atol=1e-3 if exact else 0.06)
  free = s(prompt_token_ids=prompts, max_generation_steps=8, eos_tokens=[-1])
  banned = sorted({int(t) for r in free.tokens for t in r})[:20]
  held = s(prompt_token_ids=prompts, max_generation_steps=8, eos_tokens=[-1], forbidden_tokens=banned, return_logits=True)
  assert not {int(t) for r in held.tokens for t in r} & set(banned)
  assert held.logits[0].shape == (8, 101)
  want = plain('mixed', st, np.concatenate([prompts[0], held.tokens[0]]), dtype)[8:-1]
  assert LC.error(held.logits[0], want) < LC.LIMIT[dtype]


def test_samples_of_one_prompt_and_graph_replay_agree_with_plain_decoding():
  """The cache fill shared by samples of one prompt, and recorded steps replayed, give the tokens of the plain run."""
  m, _ = model('wide', 'bfloat16')
  base = [toks('wide', 70, i) for i in range(2)]
  prompts = [p for p in base for _ in range(4)]
  s = sampler(m, 128)
  s.share_prompt_kv = False
  want = s(prompt_token_ids=prompts, max_generation_steps=20, eos_tokens=[-1])
  s.share_prompt_kv = True
  got = s(prompt_token_ids=prompts, max_generation_steps=20, eos_tokens=[-1])
  assert all((a == b).all() for a, b in zip(want.tokens, got.tokens))
  s.use_graph = True
  for _ in range(3):
    again = s(prompt_token_ids=prompts, max_generation_steps=20, eos_tokens=[-1])
    assert all((a == b).all() for a, b in zip(got.tokens, again.tokens))
    torch.cuda.synchronize()
    s.use_graph = not s.use_graph


def test_rollout_and_scoring():
  from tunix_amd.rollout import TmxRollout
  m, st = model('mixed', 'float32')
  r = TmxRollout(rollout_actor=m, tokenizer=C.ToyTokenizer(), rollout_config=RolloutConfig(kv_cache_size=64))
  prompts = [toks('mixed', 8, i + 40) for i in range(3)]
  out = r.generate(None, RolloutConfig(max_tokens_to_generate=10, temperature=1.0, top_p=1.0, seed=1, max_prompt_length=8,
                                       kv_cache_size=64, eos_tokens=[-1], return_logprobs=True), prompt_token_ids=prompts)
  lp = r.get_per_token_logps(np.stack(prompts), np.stack(out.tokens))
  ids = np.concatenate([np.stack(prompts), np.stack(out.tokens)], 1)
  if (ids != 0).all():                      # id 0 pads, and would be masked out of the scored sequence
    np.testing.assert_allclose(lp, np.stack([np.array(x) for x in out.logprobs]), atol=2e-4)
  assert r.model() is m and np.isfinite(lp).all()


@pytest.mark.parametrize('dtype', FORMATS)
def test_trace_command(dtype, tmp_path):
  from test_latent import save_model
  cfg = LC.CONFIGS['mixed']
  _, st = model('mixed', dtype)
  save_model(tmp_path / 'model', cfg, st)
  (tmp_path / 'out').mkdir()
  a, b = toks('mixed', 50, 1), toks('mixed', 20, 2)
  steps = [{'step': 0, 'entries': [{'id': 'a', 'tokens': a[:40].tolist(), 'want': [0, 31, 39]}, {'id': 'b', 'tokens': b[:18].tolist(), 'want': [17]}], 'end': []}]
  for i in range(10):
    ent = [{'id': 'a', 'tokens': [int(a[40 + i])], 'want': [0] if i % 3 == 0 else []}]
    if i < 2:
      ent.insert(0, {'id': 'b', 'tokens': [int(b[18 + i])], 'want': [0]})
    steps.append({'step': i + 1, 'entries': ent, 'end': (['b'] if i == 1 else []) + (['a'] if i == 9 else [])})
  steps.append({'step': 11, 'entries': [{'id': 'b', 'tokens': b.tolist(), 'want': [3]}], 'end': ['b']})
  root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
  p = subprocess.run([sys.executable, os.path.join(root, 'bin', 'trace_run'), '--model', str(tmp_path / 'model'), '--dtype', dtype,
                      '--out', str(tmp_path / 'out'), '--max-tokens', '80'], input='\n'.join(json.dumps(s) for s in steps) + '\n',
                     capture_output=True, text=True, timeout=100)
  assert p.returncode == 0, p.stderr[-2000:]
  assert [l for l in p.stdout.splitlines() if l.startswith('done')] == [f'done {i}' for i in range(12)]
  read = lambda n: np.fromfile(tmp_path / 'out' / f'{n}.f32', '<f4').reshape(-1, 101)
  pa, pb = plain('mixed', st, a, dtype), plain('mixed', st, b, dtype)
  assert LC.error(read(0), np.stack([pa[0], pa[31], pa[39], pb[17]])) < LC.LIMIT[dtype]
  assert LC.error(read(1), np.stack([pb[18], pa[40]])) < LC.LIMIT[dtype]
  assert LC.error(read(10), pa[49:50]) < LC.LIMIT[dtype] and LC.error(read(11), pb[3:4]) < LC.LIMIT[dtype]
  assert not (tmp_path / 'out' / '3.f32').exists()
