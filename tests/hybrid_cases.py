"""Small configurations and random weights of decoder-only models (hybrid ones and
ones with latent attention), for the tests on the CPU and on the GPU."""

import json

import numpy as np

from oracle import hybrid_lm
from oracle import latent_lm


def attention(heads, kv_heads, dim, vdim, window, scale=None):
  return {'type': 'attention', 'mixer': {
      'heads': heads, 'kv_heads': kv_heads, 'dim': dim, 'vdim': vdim,
      'mask': {'size': window}, 'scale': scale or dim ** -0.5}}


def gla(heads, dim, vdim, tau=8.0):
  return {'type': 'gla', 'mixer': {'heads': heads, 'dim': dim, 'vdim': vdim,
                                   'tau': tau}}


def delta(heads, kv_heads, dim, vdim, taps=4):
  return {'type': 'channel_delta', 'mixer': {
      'heads': heads, 'kv_heads': kv_heads, 'dim': dim, 'vdim': vdim,
      'conv': taps}}


def layer(mixer, ff=None, limit=1.5):
  return dict(mixer, mlp=None if ff is None else
              {'kind': 'dense', 'ff': ff, 'limit': limit})


def config(width, vocab, layers, loop=None, eps=1e-5):
  c = {'architecture': 'Mokivik', 'width': width, 'vocab': vocab,
       'norm': {'eps': eps}, 'layers': layers}
  if loop is not None:
    c['loop'] = dict(zip(('start', 'stop', 'times'), loop))
  return c


def latent(heads, dim, vdim, q_rank, kv_rank, window, kv_from=None, scale=None):
  m = {'heads': heads, 'dim': dim, 'vdim': vdim, 'q_rank': q_rank,
       'kv_rank': kv_rank, 'mask': {'size': window},
       'scale': scale or dim ** -0.5}
  if kv_from is not None:
    m['kv_from'] = kv_from
  return {'type': 'latent_attention', 'mixer': m}


def moe(mixer, experts, top, ff, limit, shared=None):
  return dict(mixer, mlp={
      'kind': 'moe', 'router': {'experts': experts, 'top': top},
      'expert': {'ff': ff, 'limit': limit},
      'shared': None if shared is None else dict(zip(('ff', 'limit'), shared))})


def dense(mixer, ff):
  return dict(mixer, mlp={'kind': 'dense', 'ff': ff})


def latent_config(width, vocab, layers, streams, scale=3.0, eps=1e-5):
  c = {'architecture': 'Nutizen', 'width': width, 'vocab': vocab,
       'norm': {'eps': eps}, 'embedding': {'scale': scale}, 'layers': layers}
  if streams is not None:
    c['streams'] = streams
  return c


# Sizes chosen to differ from one another and from the tiles of the kernels.
CONFIGS = {
    'all': config(88, 101, [
        layer(delta(6, 2, 24, 40, taps=4), ff=72, limit=0.7),
        layer(attention(6, 3, 40, 24, 9)),
        layer(gla(3, 20, 36, tau=5.0), ff=56, limit=2.0),
        layer(attention(5, 1, 16, 48, 33, scale=0.4), ff=136),
    ], loop=(1, 3, 2)),
    'no_loop': config(64, 130, [
        layer(attention(4, 4, 32, 32, 70)),
        layer(gla(2, 72, 12), ff=64),
        layer(delta(3, 3, 68, 16, taps=2)),
    ]),
    'all_looped': config(48, 67, [
        layer(delta(2, 1, 130, 20, taps=5)),
        layer(attention(2, 2, 70, 130, 5), ff=40),
    ], loop=(0, 2, 3)),
    'odd_values': config(40, 50, [
        layer(gla(2, 8, 10, tau=1.0)),
        layer(delta(2, 2, 8, 6, taps=1), ff=24),
        layer(attention(3, 1, 10, 6, 1)),
        layer(attention(16, 1, 8, 8, 130)),
    ], loop=(2, 3, 1)),
    'one_kind': config(72, 96, [layer(gla(4, 16, 16))], loop=(0, 1, 2)),
    'latent': latent_config(88, 101, [
        moe(latent(5, 24, 40, 56, 72, 9), 6, 2, 40, 0.8, (72, 1.1)),
        dense(latent(3, 40, 20, 48, 72, 70, scale=0.4), 104),
        moe(latent(6, 16, 16, 24, 72, 33, kv_from=0), 5, 3, 24, 2.0, (40, 0.6)),
        layer(latent(2, 36, 12, 40, 72, 5, kv_from=1)),
    ], streams=3),
    'latent_plain': latent_config(72, 60, [
        moe(latent(20, 8, 10, 20, 30, 65, scale=0.7), 4, 4, 24, 1.5),
        moe(latent(1, 70, 130, 100, 300, 1), 3, 1, 8, 0.5),
        dense(latent(4, 12, 36, 130, 30, 40, kv_from=0), 40),
    ], streams=1, scale=1.0),
    'latent_one_stream': latent_config(64, 50, [
        dense(latent(2, 300, 20, 32, 64, 12), 64),
        moe(latent(17, 6, 5, 9, 600, 130), 9, 2, 70, 1.0, (16, 0.7)),
    ], streams=None, scale=0.5, eps=1e-3),
    'latent_streams': latent_config(130, 90, [
        dense(latent(4, 32, 32, 64, 128, 64), 96),
        moe(latent(4, 32, 32, 64, 128, 2, kv_from=0), 2, 1, 64, 1.2, (64, 9.0)),
    ], streams=6),
}
LATENT = sorted(n for n in CONFIGS if n.startswith('latent'))


def forward(cfg, w, tokens, trace=None):
  """The oracle's logits."""
  lm = latent_lm if cfg['architecture'] == 'Nutizen' else hybrid_lm
  return lm.forward(cfg, w, tokens, trace)


def bf16(x):
  """Rounded to bfloat16, as float32."""
  u = np.ascontiguousarray(x, np.float32).view(np.uint32)
  return ((u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000).astype(
      np.uint32).view(np.float32)


def random_params(cfg, seed=0, ranks=(12, 7)):
  """bfloat16-valued weights by tensor name for a config dict.  Decays reach from
  a token to thousands, sinks and query / key norms are large enough to matter."""
  if cfg['architecture'] == 'Nutizen':
    return random_latent_params(cfg, seed)
  rs = np.random.RandomState(seed)
  W, V = cfg['width'], cfg['vocab']
  lin = lambda o, i: rs.randn(o, i) / np.sqrt(i)
  norm = lambda n: 1.0 + 0.3 * rs.randn(n)
  w = {'embed': rs.randn(V, W), 'final.norm': norm(W), 'head': lin(V, W)}
  if cfg.get('loop'):
    w['loop.in'] = lin(W, 2 * W)
    w['loop.step'] = rs.randn(cfg['loop']['times'], W)
  for i, l in enumerate(cfg['layers']):
    p, m = f'l{i}.', l['mixer']
    H, G, D, Dv = m['heads'], m.get('kv_heads', m['heads']), m['dim'], m['vdim']
    w[p + 'norm1'], w[p + 'norm1b'] = norm(W), norm(W)
    t = {'o': lin(W, H * Dv)}
    if l['type'] == 'attention':
      t.update({'q': lin(H * D, W), 'k': lin(G * D, W), 'v': lin(G * Dv, W),
                'q.norm': 2.0 * norm(D), 'k.norm': norm(D),
                'sink': 2.0 * rs.randn(H)})
    elif l['type'] == 'gla':
      r = ranks[0]
      t.update({'q': lin(H * D, W), 'k': lin(H * D, W), 'v': lin(H * Dv, W),
                'g': lin(H * Dv, W), 'norm': norm(Dv), 'a1': lin(r, W),
                'a2': lin(H * D, r), 'a2.b': 2.5 * rs.randn(H * D)})
    else:
      r, r2 = ranks
      taps = m['conv']
      t.update({'b': lin(H, W), 'A_log': rs.randn(H), 'norm': norm(Dv),
                'a1': lin(r, W), 'a2': lin(H * D, r),
                'dt_bias': -2.0 + 2.5 * rs.randn(H * D), 'g1': lin(r2, W),
                'g2': lin(H * Dv, r2)})
      for n, c in (('q', G * D), ('k', G * D), ('v', H * Dv)):
        t[n], t[n + '.conv'] = lin(c, W), rs.randn(c, taps)
    w.update({p + 'mix.' + k: v for k, v in t.items()})
    if l['mlp'] is not None:
      F = l['mlp']['ff']
      w[p + 'norm2'], w[p + 'norm2b'] = norm(W), norm(W)
      w[p + 'mlp.gate'], w[p + 'mlp.up'] = lin(F, W), lin(F, W)
      w[p + 'mlp.down'] = lin(W, F)
  return {k: bf16(v) for k, v in w.items()}


def random_latent_params(cfg, seed=0):
  """Scores of a few units, so that single keys matter; streams that differ."""
  rs = np.random.RandomState(seed)
  W, V, n = cfg['width'], cfg['vocab'], cfg.get('streams')
  lin = lambda o, i, gain=1.0: gain * rs.randn(o, i) / np.sqrt(i)
  norm = lambda k: 1.0 + 0.3 * rs.randn(k)
  w = {'embed': rs.randn(V, W), 'final.norm': norm(W), 'head': lin(V, W)}

  def unit(p, F):
    w[p + 'gate'], w[p + 'up'] = lin(F, W), lin(F, W)
    w[p + 'down'] = lin(W, F)

  def around(p, q):
    w[f'{p}norm{q}'] = norm(W)
    if n is not None:
      w[f'{p}hc{q}.in'] = (0.5 + rs.rand(n)) / n
      w[f'{p}hc{q}.out'] = 0.3 + rs.rand(n)
      w[f'{p}hc{q}.mix'] = 0.8 * np.eye(n) + 0.4 * rs.rand(n, n) / n

  for i, l in enumerate(cfg['layers']):
    p, m, mlp = f'l{i}.', l['mixer'], l['mlp']
    H, D, Dv, r = m['heads'], m['dim'], m['vdim'], m['kv_rank']
    around(p, 1)
    w[p + 'mix.dq'], w[p + 'mix.dq.norm'] = lin(m['q_rank'], W), norm(m['q_rank'])
    w[p + 'mix.uq'] = lin(H * D, m['q_rank'], 1.5)
    if 'kv_from' not in m:
      w[p + 'mix.dkv'], w[p + 'mix.dkv.norm'] = lin(r, W), norm(r)
    w[p + 'mix.uk'], w[p + 'mix.uv'] = lin(H * D, r, 1.5), lin(H * Dv, r)
    w[p + 'mix.sink'], w[p + 'mix.o'] = 1.5 * rs.randn(H), lin(W, H * Dv)
    if mlp is None:
      continue
    around(p, 2)
    if mlp['kind'] == 'dense':
      unit(p + 'mlp.', mlp['ff'])
      continue
    E, top = mlp['router']['experts'], mlp['router']['top']
    w[p + 'mlp.table'] = np.argsort(rs.rand(V, E), axis=1)[:, :top].astype(np.int32)
    for e in range(E):
      unit(f'{p}mlp.e{e}.', mlp['expert']['ff'])
    if mlp['shared']:
      unit(p + 'mlp.shared.', mlp['shared']['ff'])
      w[p + 'mlp.shared.sg'] = lin(1, W, 2.0)
  return {k: v if v.dtype == np.int32 else bf16(v) for k, v in w.items()}


def save_model(directory, cfg, params):
  """config.json and a bfloat16 (tables: int32) model.safetensors."""
  (directory / 'config.json').write_text(json.dumps(cfg))
  header, blobs, at = {}, [], 0
  for name, x in params.items():
    ints = x.dtype == np.int32
    blob = (x.astype('<i4') if ints else
            (np.ascontiguousarray(x, np.float32).view(np.uint32) >> 16).astype(
                '<u2')).tobytes()
    header[name] = {'dtype': 'I32' if ints else 'BF16', 'shape': list(x.shape),
                    'data_offsets': [at, at + len(blob)]}
    at += len(blob)
    blobs.append(blob)
  head = json.dumps(header).encode()
  with open(directory / 'model.safetensors', 'wb') as fp:
    fp.write(len(head).to_bytes(8, 'little') + head + b''.join(blobs))
