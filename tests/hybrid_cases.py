"""Small configurations and random weights of hybrid decoder-only models, for the
tests on the CPU and on the GPU."""

import json

import numpy as np


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
}


def bf16(x):
  """Rounded to bfloat16, as float32."""
  u = np.ascontiguousarray(x, np.float32).view(np.uint32)
  return ((u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000).astype(
      np.uint32).view(np.float32)


def random_params(cfg, seed=0, ranks=(12, 7)):
  """bfloat16-valued weights by tensor name for a config dict.  Decays reach from
  a token to thousands, sinks and query / key norms are large enough to matter."""
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


def save_model(directory, cfg, params):
  """config.json and a bfloat16 model.safetensors."""
  (directory / 'config.json').write_text(json.dumps(cfg))
  header, blobs, at = {}, [], 0
  for name, x in params.items():
    blob = (np.ascontiguousarray(x, np.float32).view(np.uint32) >> 16).astype(
        '<u2').tobytes()
    header[name] = {'dtype': 'BF16', 'shape': list(x.shape),
                    'data_offsets': [at, at + len(blob)]}
    at += len(blob)
    blobs.append(blob)
  head = json.dumps(header).encode()
  with open(directory / 'model.safetensors', 'wb') as fp:
    fp.write(len(head).to_bytes(8, 'little') + head + b''.join(blobs))
