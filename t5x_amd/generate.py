"""Generation from token ids with any registered decoder-only model: what
bin/generate runs.  Every line of standard input is a prompt, a JSON list of token
ids; every line of output is the JSON list of the tokens generated after it.
"""

import argparse
import json
import sys


def parse_args(argv=None):
  ap = argparse.ArgumentParser(
      prog='generate', description='Continue prompts of token ids (one JSON list '
      'per line of standard input).')
  ap.add_argument('--model', required=True,
                  help='folder with config.json and the weights')
  ap.add_argument('--dtype', default='bfloat16',
                  choices=['bfloat16', 'float32'])
  ap.add_argument('--tokens', type=int, default=32,
                  help='most tokens generated per prompt')
  ap.add_argument('--eos', type=int, default=1,
                  help='token that ends a sequence')
  ap.add_argument('--temperature', type=float, default=0.0)
  ap.add_argument('--topk', type=int, default=0)
  ap.add_argument('--topp', type=float, default=0.0)
  ap.add_argument('--beams', type=int, default=0,
                  help='beam search with this many beams instead of sampling')
  ap.add_argument('--batch', type=int, default=16,
                  help='prompts that decode together')
  ap.add_argument('--seed', type=int, default=0)
  return ap.parse_args(argv)


def main(argv=None):
  args = parse_args(argv)
  from t5x_amd import _lib
  _lib.ensure_built()
  import functools
  from t5x_amd import decoding
  from t5x_amd import models
  from t5x_amd import registry
  if args.beams:
    decode_fn = decoding.beam_search
  else:
    decode_fn = functools.partial(
        decoding.temperature_sample, temperature=args.temperature,
        topk=args.topk, topp=args.topp)
  model, params = registry.load_model(
      args.model, args.dtype, decode_fn=decode_fn,
      output_vocabulary=models.Vocabulary(args.eos))
  prompts = [json.loads(line) for line in sys.stdin if line.strip()]
  for tokens in model.generate(params, prompts, args.tokens,
                               batch_size=args.batch,
                               num_decodes=max(1, args.beams), seed=args.seed):
    sys.stdout.write(json.dumps(tokens) + '\n')
    sys.stdout.flush()
  return 0
