"""Models by the `architecture` name in their config.json.

`load_model(directory)` reads config.json and the weights beside it and returns
the model object (models.EncoderDecoderModel or models.DecoderOnlyModel) with its
parameters; `module_from_config` builds the module alone.  A new design is a new
entry in ARCHITECTURES.
"""

import dataclasses
import json
import os
from typing import Any, Callable, Mapping

from t5x_amd import checkpoints


@dataclasses.dataclass(frozen=True)
class Architecture:
  """make_module(config dict, dtype, device) -> module; make_model(module,
  **model arguments) -> model; load_params(directory) -> parameters."""
  make_module: Callable
  make_model: Callable
  load_params: Callable


def _t5_module(config, dtype, device):
  from t5x_amd import network
  fields = {f.name for f in dataclasses.fields(network.T5Config)}
  kw = {k: v for k, v in config.items() if k in fields and k != 'dtype'}
  if 'size' in config:
    cfg = network.t5_1_1_config(config['size'], dtype=dtype, **kw)
  else:
    cfg = network.T5Config(dtype=dtype, **kw)
  return network.Transformer(cfg, device)


def _t5_model(module, **kw):
  from t5x_amd import models
  return models.EncoderDecoderModel(module, **kw)


def _hybrid_module(config, dtype, device):
  from t5x_amd import hybrid
  return hybrid.HybridDecoder(hybrid.HybridConfig.from_dict(config, dtype),
                              device)


def _decoder_only_model(module, **kw):
  from t5x_amd import models
  return models.DecoderOnlyModel(module, **kw)


def _safetensors_params(directory):
  return checkpoints.load_safetensors(
      os.path.join(directory, 'model.safetensors'))


ARCHITECTURES = {
    'T5.1.1': Architecture(_t5_module, _t5_model, checkpoints.load_params),
    'Mokivik': Architecture(_hybrid_module, _decoder_only_model,
                            _safetensors_params),
    'Nutizen': Architecture(_hybrid_module, _decoder_only_model,
                            _safetensors_params),
}


def architecture_of(config: Mapping[str, Any]) -> Architecture:
  name = config.get('architecture')
  if name not in ARCHITECTURES:
    raise ValueError(f'unknown architecture {name!r}; known: '
                     f'{sorted(ARCHITECTURES)}')
  return ARCHITECTURES[name]


def read_config(directory: str) -> dict:
  with open(os.path.join(directory, 'config.json'), encoding='utf-8') as fp:
    return json.load(fp)


def module_from_config(config: Mapping[str, Any], dtype: str = 'bfloat16',
                       device=None):
  return architecture_of(config).make_module(config, dtype, device)


def load_model(directory: str, dtype: str = 'bfloat16', device=None,
               **model_kwargs):
  """-> (model, params)."""
  config = read_config(directory)
  arch = architecture_of(config)
  module = arch.make_module(config, dtype, device)
  return arch.make_model(module, **model_kwargs), arch.load_params(directory)
