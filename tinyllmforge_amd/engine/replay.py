"""Replays a trace of given token ids through an engine, step by step, and hands out logits instead of tokens.

A step is a batch of entries ``(request id, next tokens, wanted places)``.  It runs through the engine's own scheduler
state (blocks, state slots), model runner, caches and kernels; only the choice of the batch and of the tokens is the
trace's."""
from __future__ import annotations

from .llm_engine import LLMEngine
from .sequence import Sequence


class Replay:
    def __init__(self, engine: LLMEngine):
        if not engine.model_runner.portioned:
            raise ValueError("traces are replayed by models that run prompts in portions")
        self.engine = engine
        self.live: dict[str, Sequence] = {}

    def step(self, entries, end=()):
        """``entries``: dicts with ``id``, ``tokens``, ``want``.  Returns fp32 logits ``[wanted, vocab]`` on the host
        (None if nothing is wanted); the requests named in ``end`` give back what they hold."""
        sched, runner = self.engine.scheduler, self.engine.model_runner
        limit = self.engine.config.max_model_len
        seqs = []
        entries = [e for e in entries if e["tokens"]]
        for e in entries:
            tokens = e["tokens"]
            seq = self.live.get(e["id"])
            if seq is None:
                if len(self.live) >= self.engine.config.max_num_seqs:
                    raise RuntimeError("more live requests than the engine holds")
                seq = self.live[e["id"]] = Sequence(tokens)
            else:
                for t in tokens:
                    seq.append_token(t)
            if len(seq) > limit:
                raise RuntimeError(f"request {e['id']} is longer than max_model_len = {limit}")
            seq.num_scheduled = len(tokens)
            if not sched.can_admit(seq):
                raise RuntimeError("the KV pool or the state slots are exhausted")
            sched.admit(seq)
            seqs.append(seq)
        logits = None
        if seqs:
            logits = runner.logits_portions(seqs, [e["want"] for e in entries])
            if logits is not None:
                logits = logits.float().cpu()
            for seq in seqs:
                seq.num_computed += seq.num_scheduled
                seq.num_scheduled = 0
        for name in end:
            sched.release(self.live.pop(name))
        return logits


def replay_main(argv=None) -> int:
    import argparse
    import json
    import os
    import sys

    ap = argparse.ArgumentParser(description="Replay a trace of token ids (JSON steps on standard input) and write logits.")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True, help="tokens that live requests hold at most, in all")
    ap.add_argument("--max-requests", type=int, default=4, help="requests that are live at most")
    a = ap.parse_args(argv)

    from ..config import model_config
    if a.dtype == "float32" and not model_config(a.model).float32:
        print(f"{a.model}: this model has no 32-bit kernels", file=sys.stderr)
        return 3
    block = 64
    tokens = -(-a.max_tokens // block) * block
    engine = LLMEngine(a.model, dtype=a.dtype, kvcache_block_size=block, num_kvcache_blocks=tokens // block,
                       max_num_seqs=a.max_requests, num_state_slots=a.max_requests, max_model_len=tokens,
                       max_num_batched_tokens=tokens)
    replay = Replay(engine)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = replay.step(step["entries"], step.get("end", []))
        if logits is not None:
            part = os.path.join(a.out, f".{step['step']}.part")
            logits.contiguous().numpy().astype("<f4").tofile(part)
            os.replace(part, os.path.join(a.out, f"{step['step']}.f32"))
        print(f"done {step['step']}", flush=True)
    return 0
