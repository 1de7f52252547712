"""Decoders of parallel mixers (grouped attention within chunks beside a delta rule with channel
decays) whose layers may run in a loop, against the plain oracle: each mechanism alone, prompts,
portions, decoding, batches, re-used slots, single keys at the borders of chunks and tiles, long
memories, growing caches, and generation through the framework's own entry points."""
import json

import numpy as np
import pytest
import torch

from metaseq_amd import (Dictionary, GeneratorInterface, SequenceGenerator,
                         TransformerLanguageModel)
from metaseq_amd import generate, trace_run
from metaseq_amd.service import ContinuousBatcher
from oracle import hybrid_oracle as O
from tests import hybrid_common as H

pytestmark = pytest.mark.gpu
F32, BF16 = torch.float32, torch.bfloat16
DTYPES = pytest.mark.parametrize("dtype", [F32, BF16], ids=["f32", "bf16"])


def only(side):
    """Weights under which one side of every parallel mixer says nothing."""
    def tweak(state):
        for k, v in state.items():
            if k.endswith({"left": "right.out", "right": "left.out"}[side]):
                v.zero_()
    return tweak


ATTENTION = {
    "plain": dict(),
    "one-head": dict(heads=1, kv_heads=1, dim=64, vdim=64),
    "many-heads-per-group": dict(heads=36, kv_heads=2, dim=8, vdim=12, rot=(100.0, 8)),
    "equal-heads": dict(heads=5, kv_heads=5, dim=64, vdim=128, rot=(1e6, 64)),
    "wide": dict(heads=3, kv_heads=1, dim=130, vdim=250, rot=(1e4, 100)),
    "wide-keys": dict(heads=2, kv_heads=1, dim=250, vdim=100, rot=(1e4, 250)),
    "beyond-the-tiles": dict(heads=2, kv_heads=2, dim=260, vdim=40, rot=(1e4, 26)),
    "values-beyond-the-tiles": dict(heads=4, kv_heads=2, dim=16, vdim=270),
    "no-rotation": dict(rot=None),
    "one-pair": dict(rot=(7.0, 2)),
    "odd-pairs": dict(dim=30, rot=(3000.0, 30)),
    "no-chunks": dict(chunk=None),
    "chunks-of-one": dict(chunk=1),
    "chunks-of-two": dict(chunk=2),
    "chunks-of-a-tile": dict(chunk=64),
    "chunks-longer-than-all": dict(chunk=4096),
}
DELTA = {
    "plain": dict(),
    "one-head": dict(delta_heads=1, delta_kv_heads=1, delta_dim=7, delta_vdim=100),
    "one-tap": dict(conv=1),
    "eight-taps": dict(conv=8),
    "wide": dict(delta_heads=4, delta_kv_heads=1, delta_dim=130, delta_vdim=130),
    "keys-of-a-tile": dict(delta_heads=3, delta_kv_heads=3, delta_dim=64, delta_vdim=64),
    "keys-of-96": dict(delta_dim=90, delta_vdim=48),
    "ranks-of-one": dict(ranks=(1, 1)),
    "wide-ranks": dict(ranks=(100, 130)),
    "many-heads": dict(delta_heads=20, delta_kv_heads=10, delta_dim=16, delta_vdim=32),
}


def _alone(case, name):
    for n in (1, 19, 150):
        t = case.tokens(n, seed=n)
        want = case.want(t)
        case.check(case.run(t), want, "%s, %d tokens" % (name, n))
        case.check(case.run(t, [max(1, n - 6), 1]), want, "%s, %d tokens, decoded" % (name, n))


@DTYPES
@pytest.mark.parametrize("name", sorted(ATTENTION))
def test_attention_alone(name, dtype):
    _alone(H.Case(H.looped([(H.parallel(**ATTENTION[name]), None)]), seed=3, dtype=dtype,
                  tweak=only("left")), name)


@DTYPES
@pytest.mark.parametrize("name", sorted(DELTA))
def test_delta_rule_alone(name, dtype):
    _alone(H.Case(H.looped([(H.parallel(**DELTA[name]), None)]), seed=4, dtype=dtype,
                  tweak=only("right")), name)


@DTYPES
@pytest.mark.parametrize("name", ["feed-forward", "equal-sides", "large-eps"])
def test_other_parts_alone(name, dtype):
    """The feed-forward; both sides of one padded width (one output product); an eps that shows."""
    mixer = H.parallel(heads=4, kv_heads=2, dim=32, vdim=64, delta_heads=8, delta_kv_heads=4,
                       delta_dim=32, delta_vdim=32)
    cfg = {"feed-forward": H.looped([(H.parallel(), H.dense(333))], width=100),
           "equal-sides": H.looped([(mixer, None)] * 2, width=130),
           "large-eps": H.looped([(H.parallel(), H.dense())], eps=0.5)}[name]
    _alone(H.Case(cfg, seed=6, dtype=dtype), name)


@DTYPES
@pytest.mark.parametrize("loop", [None, (0, 1, 1), (0, 1, 3), (1, 3, 2), (0, 3, 2), (2, 3, 4),
                                  (1, 2, 1)], ids=str)
def test_loops(loop, dtype):
    """Any range of layers, any number of passes; every pass has its own cache and state."""
    layers = [(H.parallel(), None), (H.parallel(heads=4, kv_heads=1, chunk=20), H.dense(70)),
              (H.parallel(conv=2, ranks=(3, 4)), None)]
    case = H.Case(H.looped(layers, loop=loop), seed=8, dtype=dtype)
    t = case.tokens(60, seed=1)
    want, streams = case.want(t, layers=True)
    assert len(case.decoder.runs) == len(streams)
    for portions in (None, [33, 2, 1]):
        case.check(case.run(t, portions), want, "loop %s, portions %s" % (loop, portions))


@DTYPES
def test_residual_stream_after_every_run(dtype):
    case = H.Case(H.looped_mixed(), seed=5, dtype=dtype)
    t = case.tokens(90)
    _, want = case.want(t, layers=True)
    seen = {}
    case.decoder.layer_probe = lambda i, x: seen.__setitem__(i, x.double().cpu())
    case.run(t)
    assert len(seen) == len(want) == 6
    limit = {F32: 1e-5, BF16: 3e-2}[dtype]
    for i in range(len(want)):
        err = float((seen[i] - want[i]).abs().max() / want[i].abs().max())
        print("run", i, err, flush=True)
        assert err <= limit, (i, err)


@DTYPES
@pytest.mark.parametrize("portions", [[1], [2], [3, 5, 2, 7], [17, 16], [64, 1, 30, 2, 2, 90],
                                      [37], [36, 2, 35, 1], [129], [100, 100, 1]], ids=str)
def test_portions_and_decoding_equal_the_prompt(portions, dtype):
    """Portions that end in front of, at and behind the ends of chunks, and run over several."""
    case = H.Case(H.looped_mixed(), seed=7, dtype=dtype)
    t = case.tokens(230, seed=2)
    case.check(case.run(t, portions), case.want(t), "portions %s" % portions)


@DTYPES
@pytest.mark.parametrize("n", [63, 64, 65, 127, 128, 129, 256, 300])
def test_prompt_lengths_around_the_kernel_borders(n, dtype):
    case = H.Case(H.looped_mixed(), seed=9, dtype=dtype)
    t = case.tokens(n, seed=n)
    case.check(case.run(t), case.want(t), "%d tokens" % n)


@DTYPES
@pytest.mark.parametrize("lens", [(5, 40, 1, 133, 2), (1, 1, 1), (20, 17, 18), (150, 3, 150)])
def test_batch_of_unequal_requests_equals_each_alone(lens, dtype):
    """Several requests in one step, continued by a second step of other lengths (decode steps
    among them), then decoded together: every logit as if the request were alone."""
    case = H.Case(H.looped_mixed(), seed=11, dtype=dtype, tweak=H.steady)
    d = case.decoder
    more = [(1, 30, 2)[i % 3] for i in range(len(lens))]
    steps = 3
    toks = [case.tokens(a + b + steps, seed=50 + i) for i, (a, b) in enumerate(zip(lens, more))]
    want = [case.want(t) for t in toks]
    cache = d.new_slot_cache(len(lens) + 2, 256)
    slots = list(range(len(lens)))[::-1]
    got = [[] for _ in lens]
    for part in range(2):
        entries, sizes = [], []
        for i, s in enumerate(slots):
            a = 0 if part == 0 else lens[i]
            b = lens[i] if part == 0 else lens[i] + more[i]
            entries.append((s, toks[i][a:b].cuda()))
            sizes.append(b - a)
        for i, piece in enumerate(d.extend(cache, entries, want_all=True).split(sizes)):
            got[i].append(piece)
    for k in range(steps):
        last = torch.zeros(cache.batch, dtype=torch.long)
        for i, s in enumerate(slots):
            last[s] = toks[i][lens[i] + more[i] + k]
        logits = d.decode_slots(cache, last.cuda())
        for i, s in enumerate(slots):
            got[i].append(logits[s:s + 1])
    for i in range(len(lens)):
        case.check(torch.cat(got[i]), want[i], "request %d of %s" % (i, (lens,)))


@DTYPES
def test_slots_are_reused_without_a_trace_of_the_last_request(dtype):
    case = H.Case(H.looped_mixed(), seed=13, dtype=dtype)
    d, cache = case.decoder, case.decoder.new_slot_cache(3, 200)
    for round_ in range(3):
        for slot in (1, 0):
            t = case.tokens(30 + 57 * round_, seed=100 * round_ + slot)
            got = case.run(t, [len(t) - 4, 1] if round_ % 2 else None, slot, cache)
            case.check(got, case.want(t), "round %d slot %d" % (round_, slot))
            d.release_slot(cache, slot)
    # a request of one token, decoded from the first position on in a used slot
    t = case.tokens(80, seed=77)
    case.check(case.run(t, [1], 1, cache), case.want(t), "decoded from the start")


@DTYPES
def test_a_copied_slot_goes_on_like_its_source(dtype):
    case = H.Case(H.looped_mixed(), seed=14, dtype=dtype)
    d, cache = case.decoder, case.decoder.new_slot_cache(3, 150)
    t = case.tokens(140, seed=3)
    want = case.want(t)
    d.prefill_slot(cache, 0, t[:130].cuda())
    d.copy_slot(cache, 0, 2, length=130)
    for slot in (2, 0):
        got = [d.extend(cache, [(slot, t[a:b].cuda())], want_all=True)
               for a, b in ((130, 131), (131, 134), (134, 140))]
        case.check(torch.cat(got), want[130:], "slot %d" % slot)


@DTYPES
def test_caches_grow_below_at_and_beyond_a_chunk(dtype):
    """A cache keeps one chunk per layer, or less where it is smaller than a chunk."""
    case = H.Case(H.looped_mixed(), seed=16, dtype=dtype)
    d, cache = case.decoder, case.decoder.new_slot_cache(2, 10)
    t = case.tokens(220, seed=5)
    want, at, got = case.want(t), 0, []
    for room in (10, 36, 37, 38, 90, 101, 220):
        cache.grow(room)
        rows = [x["keys"].shape[2] for x in cache.layers]
        assert rows == [min(room, c) for c in (37, 100, 64, 100, 64, 1000)]
        for piece in (t[at:room - 1], t[room - 1:room]):
            if len(piece):
                got.append(d.extend(cache, [(1, piece.cuda())], want_all=True))
        at = room
    case.check(torch.cat(got), want, "growing cache")


def test_result_does_not_depend_on_slot_or_neighbours_bit_for_bit():
    """Decode steps of the same rows give the same bits in other slots and beside others."""
    case = H.Case(H.looped_mixed(), seed=15, dtype=BF16)
    d = case.decoder
    t = case.tokens(50, seed=1).cuda()
    results = []
    for slot, other in ((0, 2), (2, 1)):
        cache = d.new_slot_cache(3, 64)
        d.extend(cache, [(slot, t[:49])])
        d.extend(cache, [(other, case.tokens(20, seed=slot).cuda())])
        last = torch.full((3,), 9, dtype=torch.long, device="cuda")
        last[slot] = t[49]
        results.append(d.decode_slots(cache, last)[slot].clone())
    assert torch.equal(results[0], results[1])


# ---------------------------------------------------------------- single keys
A, B = 5, 6          # the asking and the answering token


def _answering(state, cfg, alpha=6.0):
    """Makes one unrotated query dimension of every head respond to token A and that key dimension
    to token B, so that an A sees the B in its past and hardly anything else."""
    W = {k: v.double() for k, v in state.items()}
    m = cfg["layers"][0]["mixer"]["left"]
    h = O.rms(W["embed"][[A, B]], cfg["norm"]["eps"], W["l0.norm1"])
    free = m["rot"]["dims"] if m.get("rot") else 0
    for name, row, heads in (("q", h[0], m["heads"]), ("k", h[1], m["kv_heads"])):
        w = state["l0.mix.left." + name].view(heads, m["dim"], -1)
        w[:, free] = (alpha * row / row.norm()).to(w.dtype)
        state["l0.mix.left.%s.b" % name].view(heads, m["dim"])[:, free] = 0
    state["l0.mix.left.out"].mul_(8.0)    # what attention finds dominates the logits
    state["l0.mix.right.out"].zero_()


SEEKERS = {"a": dict(heads=4, kv_heads=2, dim=64, vdim=64, rot=(1e4, 20), scale=0.3),
           "b": dict(heads=18, kv_heads=1, dim=20, vdim=100, rot=(1e4, 4), scale=0.3),
           "c": dict(heads=2, kv_heads=2, dim=128, vdim=128, rot=(1e4, 64), scale=0.3),
           "d": dict(heads=2, kv_heads=1, dim=300, vdim=20, rot=(1e4, 64), scale=0.3)}


@DTYPES
@pytest.mark.parametrize("mix", sorted(SEEKERS))
@pytest.mark.parametrize("chunk", [None, 300, 130, 64])
def test_one_key_is_found_in_its_chunk_only(mix, chunk, dtype):
    """Inside the chunk the key decides the answer, just outside it changes nothing."""
    cfg = H.looped([(H.parallel(chunk=chunk, **SEEKERS[mix]), None)])
    case = H.Case(cfg, seed=17, dtype=dtype, tweak=lambda s: _answering(s, cfg))
    n = 390
    first = 0 if chunk is None else (n - 1) // chunk * chunk    # of the last position's chunk
    places = {first, first + 1, first - 1, first + 15, first + 16, first + 31, first + 32,
              first + 63, first + 64, n - 2}
    if chunk is None:
        places |= {127, 128, 255, 256, 300}
    for at in sorted(p for p in places if 0 <= p < n - 1):
        t = case.tokens(n, seed=at)
        t[t == A] = 7
        t[t == B] = 8
        t[at], t[n - 1] = B, A
        other = t.clone()
        other[at] = 9
        want, without = case.want(t)[-1:], case.want(other)[-1:]
        gap = float((want - without).pow(2).mean().sqrt() / want.pow(2).mean().sqrt())
        assert gap > 0.5 if at >= first else gap == 0, (at, gap)
        case.check(case.run(t)[-1:], want, "key %d, prompt" % at)
        case.check(case.run(t, [n - 1, 1])[-1:], want, "key %d, decoded" % at)
        if at in (first, first - 1, 255):
            for portions in ([200, 100, 60, 2], [first + 1, n - 2 - first, 1]):
                case.check(case.run(t, portions)[-1:], want, "key %d, portions" % at)


@DTYPES
def test_a_chunk_is_left_and_entered_at_its_borders(dtype):
    """Askers on both sides of a border, with the key in front of it, in prompts, portions cut
    around the border and decode steps."""
    chunk = 48
    cfg = H.looped([(H.parallel(chunk=chunk, **SEEKERS["a"]), None)])
    case = H.Case(cfg, seed=18, dtype=dtype, tweak=lambda s: _answering(s, cfg))
    n = 4 * chunk + 5
    t = case.tokens(n, seed=3)
    t[t == A] = 7
    t[t == B] = 8
    for border in (chunk, 3 * chunk):
        t[border - 3], t[border - 1], t[border], t[border + 1] = B, A, A, A
        t[border + 5], t[border + 6] = B, A
    want = case.want(t)
    for portions in (None, [chunk - 1, 1, 1, chunk], [chunk, 1], [chunk + 1, 2 * chunk - 2, 2, 2, 60],
                     [2 * chunk + 10, 30, 5, 3, 1]):
        case.check(case.run(t, portions), want, "portions %s" % portions)


@DTYPES
def test_the_next_token_is_never_seen(dtype):
    """Token B right behind an A must not answer it (prompt, portion and packed sizes)."""
    cfg = H.looped([(H.parallel(chunk=None, **SEEKERS["a"]), None)])
    case = H.Case(cfg, seed=19, dtype=dtype, tweak=lambda s: _answering(s, cfg, alpha=2.0))
    for n in (3, 17, 64, 65, 128, 200):
        t = case.tokens(n, seed=n)
        t[t == B] = 8
        t[n - 2], t[n - 1] = A, B
        case.check(case.run(t), case.want(t), "%d tokens" % n)


@DTYPES
def test_distance_shows_in_the_rotated_dimensions(dtype):
    """Scores of the rotated dimensions alone depend on the distance: hundreds of positions from
    the start, far and near keys, prompts and decode steps."""
    def rotated(state):
        only("left")(state)
        for name in ("q", "k"):
            state["l0.mix.left.%s" % name].mul_(3.0)

    for base in (50.0, 1e6):
        cfg = H.looped([(H.parallel(heads=4, kv_heads=2, dim=32, vdim=32, chunk=None,
                                    rot=(base, 32), scale=0.2), None)])
        case = H.Case(cfg, seed=20, dtype=dtype, tweak=rotated)
        t = case.tokens(400, seed=2)
        want = case.want(t)
        for portions in (None, [380, 1]):
            case.check(case.run(t, portions), want, "base %g" % base)


# ---------------------------------------------------------------- memories
@DTYPES
def test_the_first_token_is_remembered(dtype):
    """Slow decays: hundreds of positions later (and many chunks on) the first token still shows
    in the logits, across portions and decode steps."""
    def slow(state):
        only("right")(state)
        for k, v in state.items():
            if k.endswith("A_log"):
                v.fill_(-6.0)
            if k.endswith("right.b"):
                v.mul_(0.2)

    case = H.Case(H.looped([(H.parallel(delta_dim=32), None)]), seed=21, dtype=dtype, tweak=slow)
    t = case.tokens(300, seed=4)
    want = case.want(t)
    changed = t.clone()
    changed[0] = 4 + (int(t[0]) - 3) % 90
    gap = (case.want(changed)[-1] - want[-1]).pow(2).mean().sqrt() / want.pow(2).mean().sqrt()
    assert float(gap) > 20 * H.LIMIT[F32], float(gap)
    for portions in (None, [100, 31, 2, 1], [299, 1], [32], [33]):
        case.check(case.run(t, portions), want, "%s" % portions)


@DTYPES
def test_every_key_channel_has_its_own_decay(dtype):
    """Half of the channels forget at once, the others never."""
    def split(state):
        only("right")(state)
        state["l0.mix.right.A_log"].fill_(0.0)
        state["l0.mix.right.a2"].zero_()
        bias = state["l0.mix.right.dt_bias"].view(4, 20)
        bias[:, 0::2], bias[:, 1::2] = 6.0, -9.0

    case = H.Case(H.looped([(H.parallel(), None)]), seed=22, dtype=dtype, tweak=split)
    t = case.tokens(120, seed=4)
    for portions in (None, [100, 1], [7]):
        case.check(case.run(t, portions), case.want(t), "%s" % portions)


@DTYPES
def test_taps_reach_across_portions(dtype):
    case = H.Case(H.looped([(H.parallel(conv=8), None), (H.parallel(conv=7), None)]), seed=23,
                  dtype=dtype)
    t = case.tokens(40, seed=6)
    for portions in ([1], [2], [3], [1, 2, 3, 4, 5, 6, 7, 8]):
        case.check(case.run(t, portions), case.want(t), str(portions))


@DTYPES
def test_long_decoding(dtype):
    case = H.Case(H.looped_mixed(), seed=25, dtype=dtype)
    t = case.tokens(420, seed=8)
    case.check(case.run(t, [20, 1]), case.want(t), "400 decoded tokens")


@DTYPES
def test_long_input_runs_in_portions(dtype):
    case = H.Case(H.looped_mixed(), seed=27, dtype=dtype)
    d = case.decoder
    t = case.tokens(230, seed=3)
    want = case.want(t)
    d.PORTION = 100
    cache = d.new_slot_cache(2, 230)
    case.check(d.extend(cache, [(1, t.cuda())], want_all=True), want, "in portions")


# ---------------------------------------------------------------- generation
def _greedy_oracle(case, prompt, n):
    return O.greedy(prompt, n, case.W, case.json, banned=(1, 2))


def test_greedy_generation_through_the_generator():
    case = H.Case(H.looped_mixed(), seed=29, dtype=F32, tweak=H.no_specials)
    model = TransformerLanguageModel(case.decoder)
    prompts = torch.stack([torch.cat([torch.tensor([2]), case.tokens(9, seed=i)]) for i in range(3)])
    gen = SequenceGenerator([model], Dictionary(case.cfg.vocab_size), max_len_b=45, min_len=45)
    out = gen.generate([model], {"net_input": {"src_tokens": prompts.cuda()}})["tokens"].cpu()
    for i in range(3):
        want = _greedy_oracle(case, prompts[i].tolist(), 34)
        assert out[i, 0, :44].tolist() == want[:44], i


def test_unequal_prompts_and_sampling():
    case = H.Case(H.looped_mixed(), seed=31, dtype=F32, tweak=H.no_specials)
    api = GeneratorInterface(TransformerLanguageModel(case.decoder), Dictionary(case.cfg.vocab_size))
    prompts = [case.tokens(n, seed=n).tolist() for n in (39, 4, 1)]
    for extra in (dict(), dict(logprobs=3)):
        got = api.generate(prompts, min_tokens=[6] * 3, max_tokens=[6] * 3, temperature=1.0, **extra)
        for p, beams in zip(prompts, got):
            want = _greedy_oracle(case, [2] + p, 5)[1 + len(p):]
            assert [int(x) for x in beams[0]["tokens"]][:5] == want, (p, extra)
    sampled = api.generate(prompts, min_tokens=[6] * 3, max_tokens=[6] * 3, temperature=0.7,
                           top_p=0.9, seed=5)
    assert all(1 <= len(b[0]["tokens"]) <= 6 for b in sampled)


def test_greedy_generation_through_the_continuous_batcher():
    case = H.Case(H.looped_mixed(), seed=33, dtype=F32, tweak=H.no_specials)
    api = GeneratorInterface(TransformerLanguageModel(case.decoder), Dictionary(case.cfg.vocab_size))
    for prefill_batch in (1, 3):
        engine = ContinuousBatcher(api, slots=3, capacity=64, prefill_batch=prefill_batch)
        prompts = [case.tokens(n, seed=40 + n).tolist() for n in (3, 35, 8, 30, 5)]
        replies = [engine.submit(p, max_tokens=6 + i, min_tokens=6 + i)
                   for i, p in enumerate(prompts)]
        sampled = engine.submit(prompts[0], max_tokens=4, top_p=0.8, temperature=0.9, n=2)
        for _ in range(200):
            if engine.step() == 0:
                break
        for i, (p, r) in enumerate(zip(prompts, replies)):
            record = r.get_nowait()[1]
            assert not isinstance(record, Exception), record
            want = _greedy_oracle(case, [2] + p, 5 + i)[1 + len(p):]
            assert [int(x) for x in record[0]["tokens"]][:5 + i] == want, i
        assert len(sampled.get_nowait()[1]) == 2


def test_generate_command(tmp_path, capsys):
    """A model folder through the command line, as one batch and through slots."""
    case = H.Case(H.looped_mixed(), seed=37, dtype=F32, tweak=H.no_specials)
    folder = H.model_folder(tmp_path, case.json, case.state)
    prompts = [case.tokens(n, seed=n).tolist() for n in (4, 9, 2)]
    lines = [" ".join(map(str, p)) for p in prompts]
    for extra in ([], ["--slots", "2"]):
        rc = generate.main(["--model", folder, "--dtype", "float32", "--max-tokens", "5",
                            "--min-tokens", "5"] + extra, lines=lines)
        records = [json.loads(x) for x in capsys.readouterr().out.splitlines() if x[:1] == "{"]
        assert rc == 0 and len(records) == 3
        for p, r in zip(prompts, records):
            assert r["tokens"][:4] == _greedy_oracle(case, [2] + p, 4)[1 + len(p):]


@DTYPES
def test_trace_command(tmp_path, capsys, dtype):
    """Requests replayed in portions and token by token, their slots given back and used again."""
    case = H.Case(H.looped_mixed(), seed=39, dtype=dtype)
    folder = H.model_folder(tmp_path, case.json, case.state)
    out = tmp_path / "out"
    out.mkdir()
    toks = {i: case.tokens(n, seed=n) for i, n in (("a", 70), ("b", 45), ("c", 3))}
    cuts = {"a": [33, 2, 33, 1, 1], "b": [44, 1], "c": [1, 1, 1]}
    steps, expect = [], []
    for r in ("a", "b", "c"):
        at, want = 0, case.want(toks[r])
        for k, n in enumerate(cuts[r]):
            places = [] if k == 1 and r == "a" else sorted({0, n - 1})[::-1]
            steps.append(dict(step=len(steps), end=[r] if at + n == len(toks[r]) else [],
                              entries=[dict(id=r, tokens=toks[r][at:at + n].tolist(), want=places)]))
            expect.append(want[[at + p for p in places]])
            at += n
    rc = trace_run.main(["--model", folder, "--dtype", str(dtype).split(".")[1], "--out", str(out),
                         "--max-tokens", "70"], lines=[json.dumps(s) for s in steps])
    assert rc == 0
    done = [x for x in capsys.readouterr().out.splitlines() if x.startswith("done")]
    assert done == ["done %d" % i for i in range(len(steps))]
    for s, want in zip(steps, expect):
        path = out / ("%d.f32" % s["step"])
        assert path.exists() == bool(len(want))
        if len(want):
            got = torch.from_numpy(np.fromfile(path, dtype="<f4")).view(len(want), -1)
            case.check(got, want, "step %d" % s["step"])
