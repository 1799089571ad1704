"""Replays a trace of given tokens through a model, step by step, and writes the
logits asked for: what bin/trace_run runs.

Every line of the input is one step, a JSON object
  {"step": n, "entries": [{"id": ..., "tokens": [...], "want": [...]}], "end": [...]}
with each request's next tokens, the places among them whose logits are wanted,
and the requests that are finished after the step.  A step in which something is
wanted writes <out>/<n>.f32, little-endian float32 [wanted, vocab]; after every
step a line `done <n>` is printed.
"""

import argparse
import json
import os
import sys


def parse_args(argv=None):
  ap = argparse.ArgumentParser(
      prog='trace_run', description='Replay a trace of token ids from standard '
      'input through a model and write the logits asked for.')
  ap.add_argument('--model', required=True,
                  help='folder with config.json and model.safetensors')
  ap.add_argument('--dtype', default='bfloat16',
                  choices=['bfloat16', 'float32'])
  ap.add_argument('--out', required=True, help='folder for <step>.f32 files')
  ap.add_argument('--max-tokens', type=int, default=4096,
                  help='most tokens live requests hold at any time')
  ap.add_argument('--slots', type=int, default=4,
                  help='most requests that are live at any time')
  return ap.parse_args(argv)


def replay(lines, sequences, out_dir, done):
  """Runs the steps in `lines`; done(n) is called after each."""
  for line in lines:
    if not line.strip():
      continue
    step = json.loads(line)
    logits = sequences.step(
        [(e['id'], e['tokens'], e.get('want', [])) for e in step['entries']])
    if logits is not None:
      path = os.path.join(out_dir, f'{step["step"]}.f32')
      logits.cpu().numpy().astype('<f4').tofile(path)
    for request in step.get('end', []):
      sequences.end(request)
    done(step['step'])


def main(argv=None):
  args = parse_args(argv)
  from t5x_amd import _lib
  _lib.ensure_built()
  from t5x_amd import registry
  from t5x_amd import sequences
  os.makedirs(args.out, exist_ok=True)
  model, params = registry.load_model(args.model, args.dtype)
  live = sequences.Sequences(model.module, params, args.slots, args.max_tokens)

  def done(n):
    sys.stdout.write(f'done {n}\n')
    sys.stdout.flush()

  replay(iter(sys.stdin.readline, ''), live, args.out, done)
  return 0
