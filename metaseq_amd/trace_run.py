"""Replays a trace of token ids through a model, step by step, and writes logits.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Standard input holds one JSON object per line: {"step": n, "entries": [{"id", "tokens", "want"}],
"end": [ids]}.  Every entry's tokens continue its request; ``want`` lists the places among them
whose logits go to OUT/<step>.f32 (little-endian fp32 [wanted, vocab], in the order of the entries
and of ``want``).  Requests in ``end`` give their cache slot back after the step.  A line
"done <step>" follows every step.  Nothing is sampled: the tokens are the trace's own."""
import argparse
import json
import os
import sys


class SlotPool:
    """Slots for the live requests: one cache to begin with, one more whenever all slots are
    taken."""

    def __init__(self, decoder, slots, capacity):
        self.decoder, self.slots, self.capacity = decoder, slots, capacity
        self.free, self.live = [], {}

    def slot(self, request):
        if request not in self.live:
            if not self.free:
                cache = self.decoder.new_slot_cache(self.slots, self.capacity)
                self.free = [(cache, i) for i in reversed(range(self.slots))]
            self.live[request] = self.free.pop()
        return self.live[request]

    def release(self, request):
        place = self.live.pop(request, None)
        if place is not None:
            self.decoder.release_slot(*place)
            self.free.append(place)


def run_step(decoder, pool, step, torch):
    """Runs one step's entries; returns the wanted logits in order, or None if none are wanted."""
    by_cache = {}
    for n, e in enumerate(step["entries"]):
        cache, slot = pool.slot(e["id"])
        if e["tokens"]:
            by_cache.setdefault(id(cache), (cache, []))[1].append((n, slot, e))
    parts = {}
    for cache, items in by_cache.values():
        room = max(max(0, cache.host_lens[s]) + len(e["tokens"]) for _, s, e in items)
        if room > cache.capacity:
            cache.grow(room)
        want = [e["want"] for _, _, e in items]
        logits = decoder.extend(cache, [(s, e["tokens"]) for _, s, e in items],
                                want if any(want) else None)
        at = 0
        for n, _, e in items:
            parts[n] = None if logits is None else logits[at:at + len(e["want"])]
            at += len(e["want"])
    wanted = [parts[n] for n, e in enumerate(step["entries"]) if e["want"]]
    return torch.cat(wanted) if wanted else None


def main(argv=None, lines=None):
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.split("\n\n")[0])
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder the logits are written to")
    ap.add_argument("--max-tokens", type=int, default=4096,
                    help="most tokens that live requests hold at any time")
    args = ap.parse_args(argv)

    from .csrc.build import LIBS, build
    if not os.path.exists(LIBS["hybrid"]):
        build(force=True, verbose=False, components=("hybrid",))
    import torch

    from .registry import load_model, read_config
    dtype = getattr(torch, args.dtype)
    if dtype not in read_config(args.model)[0].dtypes:
        print("trace_run: this architecture does not run in %s" % args.dtype, file=sys.stderr)
        return 3
    decoder = load_model(args.model, device="cuda", dtype=dtype).decoder
    pool = SlotPool(decoder, 4, max(1, args.max_tokens))
    with torch.no_grad():
        for line in (sys.stdin if lines is None else lines):
            if not line.strip():
                continue
            step = json.loads(line)
            logits = run_step(decoder, pool, step, torch)
            if logits is not None:
                data = logits.cpu().contiguous().numpy().astype("<f4").tobytes()
                with open(os.path.join(args.out, "%d.f32" % step["step"]), "wb") as f:
                    f.write(data)
            for request in step.get("end", ()):
                pool.release(request)
            print("done %d" % step["step"], flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
