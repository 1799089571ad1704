"""Host side of the hybrid decoder-only models (no GPU): configuration, loading,
registry, request slots, trace replay, and the oracle's mechanisms against other
ways of computing them."""

import ctypes
import io
import json
import os
import stat
import subprocess

import numpy as np
import pytest

from oracle import hybrid_lm as oracle
from tests import hybrid_cases as cases
from t5x_amd import _lib
from t5x_amd import checkpoints
from t5x_amd import hybrid
from t5x_amd import registry
from t5x_amd import sequences
from t5x_amd import trace_replay

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ---- the oracle --------------------------------------------------------------


def test_oracle_window_attention_is_masked_softmax():
  rs = np.random.RandomState(0)
  T, H, G, D, Dv, W = 13, 4, 2, 5, 3, 6
  q, k, v = rs.randn(T, H, D), rs.randn(T, G, D), rs.randn(T, G, Dv)
  sink = rs.randn(H)
  got = oracle.window_attention(q, k, v, 0.7, W, sink)
  dist = np.arange(T)[:, None] - np.arange(T)[None, :]
  for h in range(H):
    s = 0.7 * q[:, h] @ k[:, h // 2].T - 2.0 ** (-2.0 * (h + 1)) * dist
    e = np.where((dist >= 0) & (dist < W), np.exp(s), 0.0)
    want = e @ v[:, h // 2] / (e.sum(1, keepdims=True) + np.exp(sink[h]))
    np.testing.assert_allclose(got[:, h], want, rtol=1e-12)


def test_oracle_recurrences_match_their_sums():
  """Without a delta rule o_t is a decayed sum over the past; with unit decay,
  beta = 1 and orthonormal keys the delta rule reads back what it wrote."""
  rs = np.random.RandomState(1)
  T, H, D, Dv = 9, 2, 4, 3
  q, k, v = rs.randn(T, H, D), rs.randn(T, H, D), rs.randn(T, H, Dv)
  alpha = rs.rand(T, H, D)
  got = oracle.gated_linear_attention(q, k, v, alpha)
  for t in range(T):
    want = np.zeros((H, Dv))
    for s in range(t + 1):
      decay = np.prod(alpha[s + 1:t + 1], axis=0)
      want += np.sum(q[t] * decay * k[s], axis=-1)[:, None] * v[s]
    np.testing.assert_allclose(got[t], want, rtol=1e-10)
  eye = np.broadcast_to(np.eye(4)[:, None, :], (4, H, D))
  ones = np.ones((4, H, D))
  v4 = rs.randn(4, H, Dv)
  np.testing.assert_allclose(
      oracle.delta_rule(eye, eye, v4, ones, np.ones((4, H))), v4, rtol=1e-12)


def test_oracle_convolution_and_sinusoid():
  x = np.arange(12.0).reshape(6, 2)
  taps = np.array([[1.0, 10.0, 100.0], [0.0, 0.0, 1.0]])
  got = oracle.causal_conv(x, taps)
  np.testing.assert_allclose(got[:, 1], x[:, 1])
  assert got[0, 0] == 100 * x[0, 0]
  assert got[1, 0] == 100 * x[1, 0] + 10 * x[0, 0]
  assert got[4, 0] == 100 * x[4, 0] + 10 * x[3, 0] + x[2, 0]
  s = oracle.sinusoid([0, 3], 6)
  np.testing.assert_allclose(s[0], [0, 1, 0, 1, 0, 1])
  np.testing.assert_allclose(s[1, :2], [np.sin(3), np.cos(3)])
  np.testing.assert_allclose(s[1, 5], np.cos(3 * 10000 ** (-4 / 6)))


@pytest.mark.parametrize('name', sorted(cases.CONFIGS))
def test_oracle_is_causal(name):
  cfg = cases.CONFIGS[name]
  w = cases.random_params(cfg)
  tokens = np.random.RandomState(2).randint(0, cfg['vocab'], 11)
  full = cases.forward(cfg, w, tokens)
  np.testing.assert_allclose(cases.forward(cfg, w, tokens[:6]), full[:6],
                             atol=1e-9)


# ---- configuration and weights --------------------------------------------------


def test_config_from_dict():
  c = hybrid.HybridConfig.from_dict(cases.CONFIGS['all'], 'float32')
  assert (c.width, c.vocab_size, c.eps, c.dtype) == (88, 101, 1e-5, 'float32')
  assert c.layers[1].mixer.window == 9 and c.layers[1].mixer.kv_heads == 3
  assert c.layers[0].mixer.taps == 4 and c.layers[0].mlp.limit == 0.7
  assert c.layers[2].mixer.tau == 5.0 and c.layers[1].mlp is None
  assert c.runs() == [(0, None), (1, 0), (2, None), (1, 1), (2, None),
                      (3, None)]
  plain = hybrid.HybridConfig.from_dict(cases.CONFIGS['no_loop'])
  assert plain.runs() == [(0, None), (1, None), (2, None)]
  assert 'loop.in' not in plain.param_shapes()


@pytest.mark.parametrize('name', sorted(cases.CONFIGS))
def test_runs_and_shapes_agree_with_the_oracle(name):
  cfg = cases.CONFIGS[name]
  c = hybrid.HybridConfig.from_dict(cfg)
  if cfg['architecture'] == 'Mokivik':
    assert [i for i, _ in c.runs()] == [i for i, _ in oracle.layer_runs(cfg)]
  else:
    assert c.runs() == [(i, None) for i in range(len(cfg['layers']))]
  have = {k: v.shape for k, v in cases.random_params(cfg).items()}
  want = c.param_shapes()
  assert set(have) == set(want)
  for k, shape in want.items():
    assert len(shape) == len(have[k])
    assert all(s in (None, h) for s, h in zip(shape, have[k])), k


@pytest.mark.parametrize('edit, message', [
    (lambda c: c['layers'][0].update(type='other'), 'unknown mixer'),
    (lambda c: c['layers'][0]['mlp'].update(kind='routed'), 'feed-forward'),
    (lambda c: c.update(loop={'start': 2, 'stop': 2, 'times': 1}), 'loop'),
    (lambda c: c['layers'][1]['mixer'].update(kv_heads=4), 'heads'),
])
def test_config_rejects_what_it_does_not_know(edit, message):
  c = json.loads(json.dumps(cases.CONFIGS['all']))
  edit(c)
  with pytest.raises(ValueError, match=message):
    hybrid.HybridConfig.from_dict(c)


def test_safetensors_round_trip(tmp_path):
  cfg = cases.CONFIGS['one_kind']
  params = cases.random_params(cfg)
  cases.save_model(tmp_path, cfg, params)
  got = checkpoints.load_safetensors(str(tmp_path / 'model.safetensors'))
  assert set(got) == set(params)
  for k, v in params.items():
    np.testing.assert_array_equal(got[k], v)
  raw = (tmp_path / 'model.safetensors').read_bytes()
  (tmp_path / 'cut.safetensors').write_bytes(raw[:-2])
  with pytest.raises(ValueError, match='data offsets'):
    checkpoints.load_safetensors(str(tmp_path / 'cut.safetensors'))
  (tmp_path / 'bad.safetensors').write_bytes(b'\xff' * 12)
  with pytest.raises(ValueError, match='not a safetensors'):
    checkpoints.load_safetensors(str(tmp_path / 'bad.safetensors'))


def test_safetensors_integer_and_float_tables(tmp_path):
  header = {'__metadata__': {'a': 'b'},
            'i': {'dtype': 'I32', 'shape': [3], 'data_offsets': [0, 12]},
            'f': {'dtype': 'F32', 'shape': [1, 2], 'data_offsets': [12, 20]},
            'e': {'dtype': 'F32', 'shape': [0], 'data_offsets': [20, 20]}}
  head = json.dumps(header).encode()
  data = np.array([1, -2, 3], '<i4').tobytes() + np.array(
      [0.5, 2], '<f4').tobytes()
  p = tmp_path / 'x.safetensors'
  p.write_bytes(len(head).to_bytes(8, 'little') + head + data)
  got = checkpoints.load_safetensors(str(p))
  assert got['i'].tolist() == [1, -2, 3] and got['f'].tolist() == [[0.5, 2]]
  assert got['e'].shape == (0,)


def test_registry_picks_the_module_by_name(tmp_path):
  from t5x_amd import models, network
  cases.save_model(tmp_path, cases.CONFIGS['one_kind'],
                   cases.random_params(cases.CONFIGS['one_kind']))
  model, params = registry.load_model(str(tmp_path), 'float32')
  assert isinstance(model, models.DecoderOnlyModel)
  assert isinstance(model.module, hybrid.HybridDecoder)
  assert model.module.dtype == 'float32' and 'head' in params
  t5 = registry.module_from_config({'architecture': 'T5.1.1', 'size': 'small'})
  assert isinstance(t5, network.Transformer) and t5.config.num_heads == 6
  with pytest.raises(ValueError, match='unknown architecture'):
    registry.module_from_config({'architecture': 'none'})


def test_weights_report_missing_and_misshapen_tensors():
  cfg = hybrid.HybridConfig.from_dict(cases.CONFIGS['one_kind'], 'float32')
  params = cases.random_params(cases.CONFIGS['one_kind'])
  del params['l0.mix.a2.b']
  with pytest.raises(ValueError, match='a2.b.*missing'):
    hybrid.HybridWeights(cfg, params, 'cpu')
  params['l0.mix.a2.b'] = np.zeros((3,), np.float32)
  with pytest.raises(ValueError, match='a2.b.*shape'):
    hybrid.HybridWeights(cfg, params, 'cpu')


def test_struct_sizes_match_the_header(tmp_path):
  names = {'t5d_ragged': _lib.Ragged, 't5d_recurrence': _lib.Recurrence,
           't5d_window_attention': _lib.WindowAttention,
           't5d_span': _lib.Span, 't5d_grouped_dense': _lib.GroupedDense,
           't5d_route': _lib.Route, 't5d_hyper_norm': _lib.HyperNorm,
           't5d_latent_attention': _lib.LatentAttention,
           't5d_experts': _lib.Experts,
           't5d_hybrid_layer': _lib.HybridLayer,
           't5d_hybrid_run': _lib.HybridRun,
           't5d_hybrid_model': _lib.HybridModel}
  src = '#include <stdio.h>\n#include <stddef.h>\n#include "t5d.h"\nint main(void) {\n'
  for c, py in names.items():
    src += f'printf("%zu\\n", sizeof({c}));\n'
    for field, _ in py._fields_:
      src += f'printf("%zu\\n", offsetof({c}, {field}));\n'
  (tmp_path / 's.c').write_text(src + 'return 0; }\n')
  subprocess.run(['gcc', '-I', os.path.join(ROOT, 'include'), '-o',
                  str(tmp_path / 's'), str(tmp_path / 's.c')], check=True)
  got = [int(x) for x in subprocess.run(
      [str(tmp_path / 's')], check=True, capture_output=True,
      text=True).stdout.split()]
  want = []
  for py in names.values():
    want.append(ctypes.sizeof(py))
    want += [getattr(py, field).offset for field, _ in py._fields_]
  assert got == want


def test_kernel_entry_points_check_their_arguments():
  """Host-side validation: nothing is launched."""
  lib = _lib.load()
  assert lib.t5d_window_head_pad(48, 20) == 64
  assert lib.t5d_window_head_pad(10, 200) == 256
  assert lib.t5d_window_head_pad(300, 8) == 320
  assert lib.t5d_window_head_pad(2000, 8) == -1
  a, b = _lib.WindowAttention(), _lib.Ragged()
  a.H, a.G = 3, 2
  assert lib.t5d_window_attention_run(None, a, b, 0) == -1
  r = _lib.Recurrence()
  r.H = r.G = r.Dv = 1
  r.D = 513
  assert lib.t5d_recurrence_run(None, r, b, 0) == -3
  assert b'512' in lib.t5d_last_error()
  assert lib.t5d_dense(None, _lib.BF16, _lib.BF16, 16, 64, 16, 16, 32, 32, 4,
                       60, 32, 0, 0.0, 0.0, 0.0) == -1
  assert lib.t5d_hybrid_step(None, _lib.HybridModel(), b, None, 0, None) == -1


# ---- request slots and trace replay -----------------------------------------------


class FakeModule:
  """Logits = (slot, position) of the token; remembers what it was fed."""

  def __init__(self):
    self.calls = []

  def init_cache(self, slots, max_len):
    return {'slots': slots, 'max_len': max_len}

  def advance(self, params, cache, portions, want, trace=None):
    import torch
    self.calls.append([(s, p, list(t)) for s, p, t in portions])
    rows = [(s, p + k) for (s, p, _), ks in zip(portions, want) for k in ks]
    return torch.tensor(rows, dtype=torch.float32) if rows else None


def test_sequences_hand_out_and_reuse_slots():
  m = FakeModule()
  s = sequences.Sequences(m, None, 2, 10)
  got = s.step([('a', [1, 2, 3], [2, 0]), ('b', [4], [])])
  assert got.tolist() == [[0, 2], [0, 0]]
  got = s.step([('b', [5, 6], [1]), ('a', [7], [0])])
  assert got.tolist() == [[1, 2], [0, 3]]
  assert s.length('a') == 4 and s.length('b') == 3 and len(s) == 2
  with pytest.raises(RuntimeError, match='free slots'):
    s.step([('c', [1], [])])
  s.end('a')
  assert s.step([('c', [9, 9], [1])]).tolist() == [[0, 1]]
  assert s.step([('c', [], [])]) is None
  with pytest.raises(ValueError, match='beyond'):
    s.step([('b', [0] * 8, [])])
  with pytest.raises(ValueError, match='wanted'):
    s.step([('b', [0], [1])])
  with pytest.raises(ValueError, match='twice'):
    s.step([('b', [0], []), ('b', [0], [])])
  assert s.length('b') == 3  # refused steps change nothing


def test_trace_replay_writes_what_is_wanted(tmp_path):
  m = FakeModule()
  live = sequences.Sequences(m, None, 1, 100)
  steps = [
      {'step': 0, 'entries': [{'id': 'x', 'tokens': [5, 6], 'want': [1]}],
       'end': []},
      {'step': 1, 'entries': [{'id': 'x', 'tokens': [7], 'want': []}],
       'end': ['x']},
      {'step': 2, 'entries': [{'id': 'y', 'tokens': [8, 9], 'want': [0, 1]}],
       'end': ['y']},
  ]
  done = []
  trace_replay.replay(io.StringIO('\n'.join(json.dumps(s) for s in steps)), live,
                      str(tmp_path), done.append)
  assert done == [0, 1, 2]
  assert sorted(os.listdir(tmp_path)) == ['0.f32', '2.f32']
  assert np.fromfile(tmp_path / '0.f32', '<f4').tolist() == [0, 1]
  assert np.fromfile(tmp_path / '2.f32', '<f4').tolist() == [0, 0, 0, 1]
  assert m.calls == [[(0, 0, [5, 6])], [(0, 2, [7])], [(0, 0, [8, 9])]]


def test_commands_are_executable():
  for name in ('trace_run', 'generate'):
    path = os.path.join(ROOT, 'bin', name)
    assert os.stat(path).st_mode & stat.S_IXUSR
    out = subprocess.run([path, '--help'], check=True, capture_output=True,
                         text=True).stdout
    assert '--model' in out and '--dtype' in out
