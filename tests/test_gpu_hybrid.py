"""Hybrid decoders against the plain oracle: every mechanism alone and together, prompts, portions,
decoding, batches of unequal requests, re-used slots, single keys that must or must not be seen,
long memories, and generation through the framework's own entry points."""
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

ALONE = {
    "latent": [(H.latent(), None)],
    "latent-one-head": [(H.latent(heads=1, dim=64, vdim=64, kv_rank=200, q_rank=130), None)],
    "latent-many-heads": [(H.latent(heads=21, dim=8, vdim=12, kv_rank=24, q_rank=16), None)],
    "latent-wide-head": [(H.latent(heads=2, dim=130, vdim=190, kv_rank=300, q_rank=24), None)],
    "latent-wide-rank": [(H.latent(heads=2, dim=16, vdim=96, kv_rank=600, q_rank=24), None)],
    "latent-borrowed": [(H.latent(), None), (H.rglru(), None), (H.latent(kv_from=0), None),
                        (H.latent(heads=5, dim=32, vdim=32, q_rank=8, kv_from=0), None)],
    "rglru": [(H.rglru(), None)],
    "rglru-one-tap": [(H.rglru(width=40, blocks=1, conv=1), None)],
    "rglru-many-blocks": [(H.rglru(width=420, blocks=10, conv=4), None)],
    "delta": [(H.delta(), None)],
    "delta-one-head": [(H.delta(heads=1, kv_heads=1, dim=7, vdim=100, conv=2), None)],
    "delta-one-tap": [(H.delta(heads=3, kv_heads=3, dim=70, vdim=16, conv=1), None)],
    "delta-wide": [(H.delta(heads=4, kv_heads=1, dim=130, vdim=130, conv=5), None)],
    "dense": [(H.rglru(width=32, blocks=1), H.dense(250))],
    "moe": [(H.rglru(width=32, blocks=1), H.moe())],
    "moe-no-groups": [(H.rglru(width=32, blocks=1), H.moe(groups=None, experts=7, top=1))],
    "moe-no-shared": [(H.rglru(width=32, blocks=1), H.moe(shared=None, experts=70, top=6,
                                                          groups=(7, 3)))],
    "moe-all": [(H.rglru(width=32, blocks=1), H.moe(experts=4, top=4, groups=(2, 2)))],
}


@DTYPES
@pytest.mark.parametrize("name", sorted(ALONE))
def test_mechanism_alone(name, dtype):
    case = H.Case(H.config(ALONE[name]), seed=3, dtype=dtype)
    for n in (1, 19, 150):
        t = case.tokens(n, seed=n)
        want = case.want(t)
        # random routers make close calls; nothing in these models carries one to the next token
        close = 0.1 if name.startswith("moe") and dtype == BF16 else 0.0
        case.check(case.run(t), want, "%s, %d tokens" % (name, n), close)
        case.check(case.run(t, [max(1, n - 6), 1]), want, "%s, %d tokens, decoded" % (name, n),
                   close)


@DTYPES
def test_residual_stream_after_every_layer(dtype):
    case = H.Case(H.mixed(dtype), seed=5, dtype=dtype)
    t = case.tokens(40)
    _, want = case.want(t, layers=True)
    seen = {}
    case.decoder.layer_probe = lambda i, x: seen.__setitem__(i, x.double().cpu())
    case.run(t)
    limit = {F32: 1e-5, BF16: 2e-2}[dtype]
    for i in range(len(want)):
        err = float((seen[i] - want[i]).abs().max() / want[i].abs().max())
        print("layer", i, err, flush=True)
        assert err <= limit, (i, err)


@DTYPES
@pytest.mark.parametrize("portions", [[1], [2], [3, 5, 2, 7], [17, 16], [64, 1, 30, 2, 2, 90],
                                      [129], [31, 33, 32]], ids=str)
def test_portions_and_decoding_equal_the_prompt(portions, dtype):
    case = H.Case(H.mixed(dtype), seed=7, dtype=dtype)
    t = case.tokens(200, seed=2)
    case.check(case.run(t, portions), case.want(t), "portions %s" % portions)


@DTYPES
@pytest.mark.parametrize("n", [127, 128, 129, 256, 300])
def test_prompt_lengths_around_the_kernel_borders(n, dtype):
    case = H.Case(H.mixed(dtype), seed=9, dtype=dtype)
    t = case.tokens(n, seed=n)
    case.check(case.run(t), case.want(t), "%d tokens" % n)


@DTYPES
@pytest.mark.parametrize("lens", [(5, 40, 1, 133, 2), (1, 1, 1), (20, 17, 18), (150, 3, 150)])
def test_batch_of_unequal_requests_equals_each_alone(lens, dtype):
    """Several requests in one step, continued by a second step of other lengths (decode steps
    among them), then decoded together: every logit as if the request were alone."""
    case = H.Case(H.mixed(dtype), seed=11, dtype=dtype)
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
    case = H.Case(H.mixed(dtype), seed=13, dtype=dtype)
    d, cache = case.decoder, case.decoder.new_slot_cache(3, 200)
    for round_ in range(3):
        for slot in (1, 0):
            t = case.tokens(30 + 57 * round_, seed=100 * round_ + slot)
            got = case.run(t, [len(t) - 4, 1] if round_ % 2 else None, slot, cache)
            case.check(got, case.want(t), "round %d slot %d" % (round_, slot))
            d.release_slot(cache, slot)
    # a request of one token, decoded from the first position on in a used slot
    t = case.tokens(6, seed=77)
    case.check(case.run(t, [1], 1, cache), case.want(t), "decoded from the start")


def test_result_does_not_depend_on_slot_or_neighbours_bit_for_bit():
    """Decode steps of the same rows give the same bits in other slots and beside others."""
    case = H.Case(H.mixed(), seed=15, dtype=BF16)
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
    """Makes the first query dimension of every head respond to token A and the first key
    dimension to token B, so that an A sees the B in its past and hardly anything else."""
    W = {k: v.double() for k, v in state.items()}
    m = cfg["layers"][0]["mixer"]
    eps = cfg["norm"]["eps"]
    h = O.rms(W["embed"][[A, B]] * cfg["embedding"]["scale"], eps, W["l0.norm1"])
    cq = O.rms(h[0] @ W["l0.mix.dq"].T, eps, W["l0.mix.dq.norm"])
    c = O.rms(h[1] @ W["l0.mix.dkv"].T, eps, W["l0.mix.dkv.norm"])
    uq = state["l0.mix.uq"].view(m["heads"], m["dim"], -1)
    uk = state["l0.mix.uk"].view(m["heads"], m["dim"], -1)
    uq[:, 0] = (alpha * cq / cq.norm()).to(uq.dtype)
    uk[:, 0] = (alpha * c / c.norm()).to(uk.dtype)
    state["l0.norm1b"].mul_(8.0)    # what attention finds dominates the logits


@DTYPES
@pytest.mark.parametrize("mix", [dict(), dict(heads=18, dim=16, vdim=16, kv_rank=128),
                                 dict(kv_rank=250, dim=64, vdim=64)], ids=["a", "b", "c"])
def test_one_far_key_is_found_from_prompts_and_decode_steps(mix, dtype):
    cfg = H.config([(H.latent(**mix), None)], scale=8.0)
    case = H.Case(cfg, seed=17, dtype=dtype, tweak=lambda s: _answering(s, cfg))
    n = 700
    for at in (0, 1, 31, 32, 63, 64, 127, 128, 255, 256, 257, 511, 512, 650, n - 2):
        t = case.tokens(n, seed=at)
        t[t == A] = 7
        t[t == B] = 8
        t[at], t[n - 1] = B, A
        other = t.clone()
        other[at] = 9
        want = case.want(t)[-1:]
        without = case.want(other)[-1:]
        # the key shows: without it the answer is another one
        gap = float((want - without).pow(2).mean().sqrt() / want.pow(2).mean().sqrt())
        assert gap > 0.5, gap
        case.check(case.run(t)[-1:], want, "key %d, prompt" % at)
        case.check(case.run(t, [n - 1, 1])[-1:], want, "key %d, decoded" % at)
        if at in (0, 255, 512):
            case.check(case.run(t, [256, 200, 100, 100, 30, 2])[-1:], want, "key %d, portions" % at)


@DTYPES
def test_the_next_token_is_never_seen(dtype):
    """Token B right behind an A must not answer it (prompt, portion and packed sizes)."""
    cfg = H.config([(H.latent(), None)], scale=8.0)
    case = H.Case(cfg, seed=19, dtype=dtype, tweak=lambda s: _answering(s, cfg, alpha=2.0))
    for n in (3, 17, 64, 65, 128, 200):
        t = case.tokens(n, seed=n)
        t[t == B] = 8
        t[n - 2], t[n - 1] = A, B
        case.check(case.run(t), case.want(t), "%d tokens" % n)


# ---------------------------------------------------------------- memories
@DTYPES
@pytest.mark.parametrize("kind", ["rglru", "delta"])
def test_the_first_token_is_remembered(kind, dtype):
    """Slow decays: hundreds of positions later the first token still shows in the logits, across
    portions and decode steps."""
    def slow(state):
        for k, v in state.items():
            if k.endswith("mix.lam"):
                v.fill_(-9.0)
            if k.endswith("mix.A_log"):
                v.fill_(-6.0)
            if k.endswith("mix.b") and v.dim() == 2:
                v.mul_(0.2)

    mixer = H.rglru(width=64, blocks=2) if kind == "rglru" else H.delta(dim=32)
    case = H.Case(H.config([(mixer, None)]), seed=21, dtype=dtype, tweak=slow)
    t = case.tokens(300, seed=4)
    want = case.want(t)
    changed = t.clone()
    changed[0] = 4 + (int(t[0]) - 3) % 90
    gap = (case.want(changed)[-1] - want[-1]).pow(2).mean().sqrt() / want.pow(2).mean().sqrt()
    assert float(gap) > 20 * H.LIMIT[F32], float(gap)
    for portions in (None, [100, 31, 2, 1], [299, 1], [32], [33]):
        case.check(case.run(t, portions), want, "%s %s" % (kind, portions))


@DTYPES
def test_taps_reach_across_portions(dtype):
    """Convolutions of many taps with portions shorter than the taps."""
    case = H.Case(H.config([(H.rglru(conv=8), None), (H.delta(conv=7), None)]), seed=23, dtype=dtype)
    t = case.tokens(40, seed=6)
    for portions in ([1], [2], [3], [1, 2, 3, 4, 5, 6, 7, 8]):
        case.check(case.run(t, portions), case.want(t), str(portions))


@DTYPES
def test_long_decoding(dtype):
    case = H.Case(H.mixed(dtype), seed=25, dtype=dtype)
    t = case.tokens(420, seed=8)
    case.check(case.run(t, [20, 1]), case.want(t), "400 decoded tokens")


@DTYPES
def test_long_input_runs_in_portions(dtype):
    case = H.Case(H.mixed(dtype), seed=27, dtype=dtype)
    d = case.decoder
    t = case.tokens(230, seed=3)
    want = case.want(t)
    d.PORTION = 100
    cache = d.new_slot_cache(2, 230)
    case.check(d.extend(cache, [(1, t.cuda())], want_all=True), want, "in portions")
    cache = d.new_slot_cache(2, 230)
    places = [229, 3, 100, 99]
    got = d.extend(cache, [(0, t[:60].cuda()), (1, t.cuda())], [[59, 0], places])
    case.check(got, torch.cat([want[[59, 0]], want[places]]), "places out of order")


# ---------------------------------------------------------------- generation
def _greedy_oracle(case, prompt, n):
    return O.greedy(prompt, n, case.W, case.json, banned=(1, 2))


def test_greedy_generation_through_the_generator():
    case = H.Case(H.mixed(), seed=29, dtype=F32, tweak=H.no_specials)
    model = TransformerLanguageModel(case.decoder)
    prompts = torch.stack([torch.cat([torch.tensor([2]), case.tokens(9, seed=i)]) for i in range(3)])
    gen = SequenceGenerator([model], Dictionary(case.cfg.vocab_size), max_len_b=25, min_len=25)
    out = gen.generate([model], {"net_input": {"src_tokens": prompts.cuda()}})["tokens"].cpu()
    for i in range(3):
        want = _greedy_oracle(case, prompts[i].tolist(), 14)
        assert out[i, 0, :24].tolist() == want[:24], i


def test_right_padded_prompts_and_nucleus_path():
    """Unequal prompts in one generator batch (pads are neither stored nor stepped); the general
    path (recorded distributions) chooses the same greedy tokens."""
    case = H.Case(H.mixed(), seed=31, dtype=F32, tweak=H.no_specials)
    api = GeneratorInterface(TransformerLanguageModel(case.decoder), Dictionary(case.cfg.vocab_size))
    prompts = [case.tokens(n, seed=n).tolist() for n in (9, 4, 1)]
    for extra in (dict(), dict(logprobs=3)):
        got = api.generate(prompts, min_tokens=[6] * 3, max_tokens=[6] * 3, temperature=1.0, **extra)
        for p, beams in zip(prompts, got):
            want = _greedy_oracle(case, [2] + p, 5)[1 + len(p):]
            assert [int(x) for x in beams[0]["tokens"]][:5] == want, (p, extra)
    sampled = api.generate(prompts, min_tokens=[6] * 3, max_tokens=[6] * 3, temperature=0.7,
                           top_p=0.9, seed=5)
    assert all(1 <= len(b[0]["tokens"]) <= 6 for b in sampled)


def test_greedy_generation_through_the_continuous_batcher():
    case = H.Case(H.mixed(), seed=33, dtype=F32, tweak=H.no_specials)
    api = GeneratorInterface(TransformerLanguageModel(case.decoder), Dictionary(case.cfg.vocab_size))
    for prefill_batch in (1, 3):
        engine = ContinuousBatcher(api, slots=3, capacity=64, prefill_batch=prefill_batch)
        prompts = [case.tokens(n, seed=40 + n).tolist() for n in (3, 17, 8, 30, 5)]
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
    case = H.Case(H.mixed(), seed=37, dtype=F32, tweak=H.no_specials)
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
    case = H.Case(H.mixed(dtype), seed=39, dtype=dtype)
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


def test_errors_are_raised_on_the_host():
    case = H.Case(H.mixed(), seed=35, dtype=BF16)
    d = case.decoder
    cache = d.new_slot_cache(2, 10)
    with pytest.raises(ValueError, match="do not fit"):
        d.extend(cache, [(0, case.tokens(11).cuda())])
    with pytest.raises(ValueError, match="slot 2"):
        d.extend(cache, [(2, case.tokens(3).cuda())])
    with pytest.raises(ValueError, match="named twice"):
        d.extend(cache, [(0, case.tokens(3).cuda()), (0, case.tokens(3).cuda())])
    with pytest.raises(ValueError, match="outside the entry"):
        d.extend(cache, [(0, case.tokens(3).cuda())], [[3]])
    d.extend(cache, [(0, case.tokens(10).cuda())])
    with pytest.raises(ValueError, match="full"):
        d.decode_slots(cache, torch.zeros(2, dtype=torch.long, device="cuda"))
