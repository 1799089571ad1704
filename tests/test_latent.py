"""Host side of the decoder-only models with latent attention (no GPU):
configuration, caches, spans, argument checks, and the oracle's mechanisms against
other ways of computing them."""

import json

import numpy as np
import pytest

from oracle import latent_lm as oracle
from tests import hybrid_cases as cases
from t5x_amd import _lib
from t5x_amd import hybrid


# ---- the oracle --------------------------------------------------------------


@pytest.mark.parametrize('window', [None, 1, 5])
def test_oracle_attention_is_masked_softmax_with_a_sink(window):
  rs = np.random.RandomState(0)
  T, H, D, Dv = 12, 3, 5, 4
  q, k, v = rs.randn(T, H, D), rs.randn(T, H, D), rs.randn(T, H, Dv)
  sink = rs.randn(H)
  got = oracle.sink_window_attention(q, k, v, 0.6, window, sink)
  dist = np.arange(T)[:, None] - np.arange(T)[None, :]
  seen = (dist >= 0) & (dist < (window or T))
  for h in range(H):
    e = np.where(seen, np.exp(0.6 * q[:, h] @ k[:, h].T), 0.0)
    want = e @ v[:, h] / (e.sum(1, keepdims=True) + np.exp(sink[h]))
    np.testing.assert_allclose(got[:, h], want, rtol=1e-12)


def test_oracle_streams():
  rs = np.random.RandomState(1)
  x, y = rs.randn(3, 4, 5), rs.randn(4, 5)
  np.testing.assert_allclose(oracle.collect(x, np.array([0, 1, 0])), x[1])
  np.testing.assert_allclose(oracle.spread(x, np.eye(3), np.ones(3), y), x + y)
  mix = np.zeros((3, 3))
  mix[0, 2] = 2.0  # from stream 0 to stream 2
  got = oracle.spread(x, mix, np.array([0.0, 1.0, 0.0]), y)
  np.testing.assert_allclose(got[2], 2 * x[0])
  np.testing.assert_allclose(got[1], y)
  assert not got[0].any()


def test_oracle_experts_follow_the_table():
  rs = np.random.RandomState(2)
  W, F, E = 6, 5, 3
  w = {f'e{e}.{n}': rs.randn(*s) for e in range(E)
       for n, s in (('gate', (F, W)), ('up', (F, W)), ('down', (W, F)))}
  w['table'] = np.array([[0, 2], [1, 0]])
  m = {'expert': {'limit': 0.4}}
  h = rs.randn(3, W)
  got = oracle.table_experts(h, [1, 0, 1], m, w.__getitem__)
  one = lambda n, e: oracle.clamped_glu(h[n], 0.4, lambda k: w[f'e{e}.{k}'])
  np.testing.assert_allclose(got[1], 0.5 * (one(1, 0) + one(1, 2)))
  np.testing.assert_allclose(got[2], 0.5 * (one(2, 1) + one(2, 0)))
  g, u = 1.3, -7.0
  unit = oracle.clamped_glu(np.array([1.0]), 0.5, {
      'gate': np.array([[g]]), 'up': np.array([[u]]),
      'down': np.array([[1.0]])}.__getitem__)
  np.testing.assert_allclose(unit, 0.5 / (1 + np.exp(-1.702 * 0.5)) * 0.5)


# ---- configuration --------------------------------------------------------------


def test_config_from_dict():
  c = hybrid.HybridConfig.from_dict(cases.CONFIGS['latent'], 'float32')
  assert (c.streams, c.hyper, c.embed_scale, c.loop) == (3, True, 3.0, None)
  a, b, r, last = c.layers
  assert a.experts.top == 2 and a.experts.shared.limit == 1.1 and not a.dense
  assert b.dense == hybrid.FeedForwardConfig(104, float('inf'), 1.0, 0.0)
  assert r.mixer.kv_from == 0 and r.experts.experts == 5 and last.mlp is None
  # a ring serves the widest window that reads it
  assert [l.mixer.reach for l in c.layers[:2]] == [33, 70]
  assert c.span_windows() == [5, 9, 33, 70]
  shapes = c.param_shapes()
  assert 'l2.mix.dkv' not in shapes and 'l3.hc2.in' not in shapes
  plain = hybrid.HybridConfig.from_dict(cases.CONFIGS['latent_one_stream'])
  assert (plain.streams, plain.hyper) == (1, False)


@pytest.mark.parametrize('edit, message', [
    (lambda c: c['layers'][2]['mixer'].update(kv_from=3), 'latents'),
    (lambda c: c['layers'][3]['mixer'].update(kv_from=2), 'latents'),
    (lambda c: c['layers'][0]['mixer'].update(kv_rank=71), 'latents'),
    (lambda c: c['layers'][0]['mlp']['router'].update(top=7), 'experts'),
    (lambda c: c['layers'][1]['mlp'].update(kind='other'), 'feed-forward'),
    (lambda c: c.update(loop={'start': 0, 'stop': 1, 'times': 2}), 'loop'),
    (lambda c: c.update(architecture='Mokivik'), None),
])
def test_config_rejects_what_it_does_not_know(edit, message):
  c = json.loads(json.dumps(cases.CONFIGS['latent']))
  edit(c)
  with pytest.raises((ValueError, KeyError), match=message):
    hybrid.HybridConfig.from_dict(c)


def test_caches_hold_latents_once():
  cfg = hybrid.HybridConfig.from_dict(cases.CONFIGS['latent'], 'float32')
  module = hybrid.HybridDecoder(cfg, 'cpu')
  module.max_portion = 10
  tree = module.init_cache(3, 200)['decoder']
  # 9 and 33 positions back, portions of 10; 70 back
  assert tree['run_0']['latent_ring'].shape == (3, 64, 128)
  assert tree['run_1']['latent_ring'].shape == (3, 128, 128)
  assert sorted(tree) == ['run_0', 'run_1']
  assert module.cache_bytes(3, 200) == 3 * (64 + 128) * 128 * 4
  portions = [(0, 0, [1] * 60)]
  assert module._portion_limit({'decoder': tree}, portions) == 64 - 33 + 1


def test_spans_cover_what_the_queries_see():
  portions = [(2, 0, [7] * 300), (0, 130, [7] * 60), (1, 63, [7] * 2)]
  p = hybrid.Portions(portions, [0, 131], 'cpu', windows=[1, 9, 0])
  spans = {s.window: s for s in p._spans}
  at = lambda ptr: (ptr - p.data.data_ptr()) // 4
  data = p.data.numpy()
  assert p.ragged.n_spans == 3 and set(spans) == {0, 1, 9}
  for window, s in spans.items():
    off = data[at(s.off):at(s.off) + 4]
    first = data[at(s.first):at(s.first) + 3]
    assert s.rows == off[-1] and off[0] == 0
    for n, (_, start, toks) in enumerate(portions):
      end = first[n] + off[n + 1] - off[n]
      assert first[n] % 64 == 0 and end % 64 == 0
      seen = max(0, start - window + 1) if window else 0
      assert seen - 63 <= first[n] <= seen
      assert start + len(toks) <= end < start + len(toks) + 64
  assert data[at(p.want_ptr):at(p.want_ptr) + 2].tolist() == [0, 131]
  # single tokens, and few beside their window, attend to the latents themselves
  assert hybrid.Portions([(0, 500, [1] * 2)], [], 'cpu', [200]).ragged.n_spans == 0
  assert hybrid.Portions([(0, 64, [1])], [], 'cpu', [1]).ragged.n_spans == 0


def test_sizes_and_argument_checks():
  lib = _lib.load()
  assert [lib.t5d_latent_pad(n) for n in (1, 65, 256, 257, 513, 1024, 1025)] == [
      128, 128, 256, 512, 576, 1024, -1]
  assert lib.t5d_grouped_tile_rows(_lib.F32, 1000, 2) == 8
  assert [lib.t5d_grouped_tile_rows(_lib.BF16, n, 4) for n in
          (3, 64, 65, 256, 257)] == [16, 16, 64, 64, 256]
  assert lib.t5d_route_max_tiles(100, 4, 16) == 6 + 4
  assert lib.t5d_route_max_tiles(3, 40, 16) == 3
  # (every count of tiles that can happen fits)
  rs = np.random.RandomState(0)
  for _ in range(200):
    n, e, rows = rs.randint(1, 300), rs.randint(1, 20), int(rs.choice([8, 16, 64]))
    counts = np.bincount(rs.randint(0, e, n), minlength=e)
    assert np.sum(-(-counts // rows)) <= lib.t5d_route_max_tiles(n, e, rows)
  b = _lib.Ragged()
  assert lib.t5d_latent_attention_run(None, _lib.LatentAttention(), b, 0) == -1
  assert lib.t5d_grouped_dense_run(None, _lib.GroupedDense()) == -1
  h = _lib.HyperNorm()
  h.x, h.streams, h.d, h.ld = 16, 17, 8, 8
  assert lib.t5d_hyper_norm_run(None, h, 1) == -3
  assert b'16' in lib.t5d_last_error()
  r = _lib.Route()
  r.experts = 2000
  assert lib.t5d_route_tokens(None, 16, 1, 1, r, 1) == -3
