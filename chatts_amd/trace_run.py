"""Replays a trace: token ids in, logits out, on the model, cache and kernels that generation uses.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Standard input carries one step per line:
    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": ["b"]}
All entries of a step run as ONE batch (SlotModel.step_tokens); a request takes a sequence slot at its first entry and gives it and its cache
pages back at the end of the step that names it in "end".  For a step in which logits are wanted, OUT/<step>.f32 holds them in the order of
the entries and of "want" (little-endian float32, [wanted, vocab]); after every step the line `done <step>` is printed.

The cache pool holds --max-tokens tokens in pages of 64; --slots sequences may be live at a time.
"""
import argparse
import json
import os
import sys

PAGE = 64


class Replay:
    """requests of a trace -> slots of a model"""

    def __init__(self, model, slots):
        self.model, self.free, self.slot_of = model, list(range(slots))[::-1], {}

    def step(self, entries, end):
        """-> logits [wanted, vocab] (float32 tensor; empty when nothing is wanted)"""
        batch = []
        for e in entries:
            if e["id"] not in self.slot_of:
                if not self.free:
                    raise RuntimeError(f"request {e['id']}: all {len(self.slot_of)} slots are taken")
                self.slot_of[e["id"]] = self.free.pop()
            want = e.get("want") or []
            if any(not 0 <= w < len(e["tokens"]) for w in want):
                raise ValueError(f"request {e['id']}: wants places outside its {len(e['tokens'])} tokens")
            batch.append((self.slot_of[e["id"]], e["tokens"], want))
        logits = self.model.step_tokens(batch)
        for rid in end:
            slot = self.slot_of.pop(rid, None)
            if slot is not None:
                self.model.release_slot(slot)
                self.free.append(slot)
        return logits


def open_model(path, dtype, max_tokens, slots, max_rows):
    from . import build, registry
    build.build()                                    # compiles on the first call of a fresh checkout, checks a stamp afterwards
    config = registry.load_config(path)
    cls = registry.model_class(config)
    pages = max(1, -(-max_tokens // PAGE))
    kw = dict(max_ctx=pages * PAGE, max_batch=slots, kv_block_size=PAGE, kv_pool_blocks=pages, max_prefill_tokens=min(max_rows, pages * PAGE))
    if getattr(config, "architecture", None) is not None:
        kw["dtype"] = dtype
    elif dtype == "float32":
        raise ValueError("ChatTS / Qwen checkpoints run with bf16 hi + lo operands; float32 is available for the designs config.json names")
    return cls.from_pretrained(path, **kw)


def main(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run", description="replay a trace of token ids and write logits")
    ap.add_argument("--model", required=True, help="directory with config.json and *.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16", help="float32: every product and sum in 32-bit")
    ap.add_argument("--out", required=True, help="directory of the <step>.f32 files")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold at any time, each rounded up to 64")
    ap.add_argument("--slots", type=int, default=4, help="sequences that may be live at a time")
    ap.add_argument("--max-rows", type=int, default=4096, help="rows of one pass; a larger step runs in several")
    a = ap.parse_args(argv)
    model = open_model(a.model, a.dtype, a.max_tokens, a.slots, a.max_rows)
    replay = Replay(model, a.slots)
    for line in sys.stdin:
        line = line.strip()
        if not line:
            continue
        s = json.loads(line)
        logits = replay.step(s["entries"], s.get("end") or [])
        if logits.shape[0]:
            data = logits.float().cpu().numpy().astype("<f4").tobytes()
            part = os.path.join(a.out, f".{s['step']}.part")
            with open(part, "wb") as f:
                f.write(data)
            os.replace(part, os.path.join(a.out, f"{s['step']}.f32"))
        print(f"done {s['step']}", flush=True)
    return 0
