"""Command line: `python -m tunix_amd generate | trace`.

generate   samples completions of prompts given as token ids with the model of a folder
           (config.json + model.safetensors) and prints one JSON line per prompt
trace      replays recorded token streams from standard input (one JSON step a line) and writes the
           wanted logits of step n to <out>/<n>.f32
"""
from __future__ import annotations

import argparse
import json
import os
import sys

DTYPES = ("bfloat16", "float32")


def _dtype(name: str):
  import torch
  return {"bfloat16": torch.bfloat16, "float32": torch.float32}[name]


def _load(args):
  """The model, or exit code 3 when its architecture does not run in the dtype asked for."""
  from . import registry
  arch, _ = registry.read_config(args.model)
  if _dtype(args.dtype) not in arch.dtypes:
    print(f"this architecture does not run in {args.dtype}", file=sys.stderr)
    raise SystemExit(3)
  return registry.load_model(args.model, args.device, _dtype(args.dtype))


def generate(args) -> int:
  from .generate import CacheConfig, Sampler
  from .generate.utils import IdTokenizer
  model = _load(args)
  tok = IdTokenizer(model.cfg.vocab_size, pad_id=args.pad_id, eos_id=args.eos[0] if args.eos else -1)
  prompts = [tok.encode(p) for p in args.prompt]
  from .generate.utils import next_power_of_2
  width = args.max_prompt_length or next_power_of_2(max(len(p) for p in prompts))
  sampler = Sampler(model, tok, CacheConfig(width + args.max_tokens))
  out = sampler(prompts, args.max_tokens, max_prompt_length=width, temperature=args.temperature, top_p=args.top_p,
                top_k=args.top_k, seed=args.seed, eos_tokens=args.eos or [-1], return_logprobs=args.logprobs)
  for i, t in enumerate(out.tokens):
    line = {"prompt": prompts[i], "tokens": [int(x) for x in t]}
    if args.logprobs:
      line["logprobs"] = [float(x) for x in out.logprobs[i]]
    print(json.dumps(line), flush=True)
  return 0


def trace(args) -> int:
  from .generate.replay import Replay
  replay = Replay(_load(args))
  for line in sys.stdin:
    if not line.strip():
      continue
    step = json.loads(line)
    logits = replay.step(step)
    if logits is not None:
      path = os.path.join(args.out, f"{int(step['step'])}.f32")
      with open(path, "wb") as f:
        f.write(logits.astype("<f4").tobytes())
    print(f"done {int(step['step'])}", flush=True)
  return 0


def main(argv=None) -> int:
  ap = argparse.ArgumentParser(prog="tunix_amd", description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
  sub = ap.add_subparsers(dest="command", required=True)
  common = argparse.ArgumentParser(add_help=False)
  common.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
  common.add_argument("--dtype", choices=DTYPES, default="bfloat16")
  common.add_argument("--device", default="cuda:0")
  g = sub.add_parser("generate", parents=[common], help="sample completions of token-id prompts")
  g.add_argument("--prompt", action="append", required=True, help='token ids, e.g. "5 17 3"; may be repeated')
  g.add_argument("--max-tokens", type=int, default=64)
  g.add_argument("--max-prompt-length", type=int, default=None)
  g.add_argument("--temperature", type=float, default=0.0)
  g.add_argument("--top-p", type=float, default=None, help="switches sampling on; without it decoding is greedy")
  g.add_argument("--top-k", type=int, default=None)
  g.add_argument("--seed", type=int, default=None)
  g.add_argument("--eos", type=int, action="append", default=None, help="end-of-sequence id; may be repeated")
  g.add_argument("--pad-id", type=int, default=-1)
  g.add_argument("--logprobs", action="store_true")
  g.set_defaults(run=generate)
  t = sub.add_parser("trace", parents=[common], help="replay recorded token streams and write logits")
  t.add_argument("--out", required=True, help="folder for <step>.f32")
  t.add_argument("--max-tokens", type=int, default=0,
                 help="most tokens that live requests hold at a time (the cache grows as needed)")
  t.set_defaults(run=trace)
  args = ap.parse_args(argv)
  return args.run(args)
