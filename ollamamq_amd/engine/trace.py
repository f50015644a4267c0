"""Trace replay: given tokens through the engine, step by step.

A thin driver over the parts that generation uses: the model registry, the
cache for the model, and LlamaEngine.feed.  Nothing is sampled.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

import torch

from ..models import build_model, config_from_folder
from .engine import LlamaEngine
from .kvcache import cache_for_model

DTYPES = {"bfloat16": torch.bfloat16, "float32": torch.float32}
MAX_LIVE = 4
PAGE = 16


def make_engine(model_dir: str, dtype: torch.dtype, max_tokens: int,
                device: str) -> LlamaEngine:
    cfg = config_from_folder(model_dir)
    pages = max(1, -(-max_tokens // PAGE))
    model = build_model(cfg, device=device, dtype=dtype)
    kv = cache_for_model(cfg, page_size=PAGE, n_pages=pages,
                         max_slots=MAX_LIVE,
                         max_ctx=min(pages * PAGE, cfg.max_ctx),
                         device=device, dtype=dtype)
    return LlamaEngine(model, kv, max_batch=MAX_LIVE)


class Replay:
    def __init__(self, engine: LlamaEngine, out_dir: str):
        self.eng = engine
        self.out_dir = out_dir
        self.live = {}

    def step(self, msg: dict) -> None:
        parts = []
        for e in msg["entries"]:
            if e["id"] not in self.live:
                self.live[e["id"]] = self.eng.open_stream()
            parts.append((self.live[e["id"]], e["tokens"],
                          e.get("want") or []))
        if parts:
            logits = self.eng.feed(parts)
            if logits.shape[0]:
                path = os.path.join(self.out_dir, f"{msg['step']}.f32")
                logits.float().cpu().numpy().astype("<f4").tofile(path)
        for rid in msg.get("end") or []:
            self.eng.close_stream(self.live.pop(rid))


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run")
    ap.add_argument("--model", required=True,
                    help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", required=True, choices=sorted(DTYPES))
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="cache size: most tokens that live requests hold")
    ap.add_argument("--device", default="cuda:0")
    args = ap.parse_args(argv)
    if args.device.startswith("cuda"):
        # a fresh checkout has no compiled kernels
        from ..build import build_kernels
        build_kernels()
    replay = Replay(make_engine(args.model, DTYPES[args.dtype],
                                args.max_tokens, args.device), args.out)
    for line in sys.stdin:
        if not line.strip():
            continue
        msg = json.loads(line)
        replay.step(msg)
        print(f"done {msg['step']}", flush=True)
    return 0
