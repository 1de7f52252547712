"""Decoders of parallel mixers in loops without a GPU: configuration, weights by name and shape,
the order of runs, what a cache keeps, and hand-computed pins of the oracle's mechanisms."""
import json
import math

import pytest
import torch

from metaseq_amd import HybridConfig, random_hybrid_state_dict, registry
from metaseq_amd.config import LoopSpec, ParallelSpec, SquaredReluSpec
from metaseq_amd.hybrid_decoder import HybridDecoder
from oracle import hybrid_oracle as O
from tests import hybrid_common as H

F64 = torch.float64


# ---------------------------------------------------------------- configuration
def test_config_reads_both_sides_and_the_loop():
    cfg = HybridConfig.from_json(H.looped_mixed())
    m = cfg.layers[2].mixer
    assert isinstance(m, ParallelSpec)
    assert (m.left.heads, m.left.kv_heads, m.left.dim, m.left.vdim) == (18, 1, 16, 20)
    assert (m.left.rot_base, m.left.rot_dims, m.left.chunk, m.left.scale) == (1e5, 6, 64, 0.25)
    assert (m.right.heads, m.right.kv_heads, m.right.conv) == (6, 1, 3)
    assert isinstance(cfg.layers[0].mlp, SquaredReluSpec) and cfg.layers[1].mlp is None
    assert cfg.loop == LoopSpec(1, 3, 2) and cfg.tied
    assert not cfg.post_norms and not cfg.sinusoidal and cfg.embed_scale == 1.0
    shapes = cfg.tensor_shapes()
    assert shapes["loop.step"] == (2, 72) and "head" not in shapes
    assert shapes["l0.mix.left.q"] == (144, 72) and shapes["l0.mix.left.v.b"] == (80,)
    assert shapes["l2.mix.right.a2"] == (120, 5) and shapes["l2.mix.right.dt_bias"] == (120,)
    assert shapes["l1.mix.right.g2"] == (48, 7) and shapes["l1.mix.right.out"] == (72,)
    assert shapes["l3.mlp.up.b"] == (200,) and "l1.norm2" not in shapes
    assert not any(n.endswith(("norm1b", "norm2b")) for n in shapes)


def test_optional_sections():
    cfg = HybridConfig.from_json(H.looped([(H.parallel(chunk=None, rot=None), None)]))
    left = cfg.layers[0].mixer.left
    assert left.chunk is None and left.rot_dims == 0 and cfg.loop is None
    assert "loop.step" not in cfg.tensor_shapes()
    c = H.looped([(H.parallel(), None)])
    c["layers"][0]["mixer"]["left"].update(mask=None, rot=None)
    c["loop"] = None
    left = HybridConfig.from_json(c).layers[0].mixer.left
    assert left.chunk is None and left.rot_dims == 0


@pytest.mark.parametrize("break_it,match", [
    (lambda c: c["layers"][0].update(type="delta"), "unknown mixer"),
    (lambda c: c["layers"][0]["mixer"]["left"].pop("scale"), "scale"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=4), "multiple of kv_heads"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(kv_heads=3), "multiple of kv_heads"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=5), "rotary"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=26), "rotary"),
    (lambda c: c["layers"][0]["mixer"]["left"]["mask"].update(size=-2), "chunks of"),
    (lambda c: c["loop"].update(stop=5), "loop of layers"),
    (lambda c: c["loop"].update(start=3), "loop of layers"),
    (lambda c: c["loop"].update(times=0), "loop of layers"),
    (lambda c: c["loop"].pop("times"), "times"),
])
def test_bad_configurations_are_refused(break_it, match):
    c = json.loads(json.dumps(H.looped_mixed()))
    break_it(c)
    with pytest.raises((ValueError, NotImplementedError), match=match):
        HybridConfig.from_json(c)


def test_unknown_keys_are_reported_not_fatal(caplog):
    c = H.looped([(H.parallel(), None)])
    c["layers"][0]["mixer"]["left"]["rot"]["twist"] = 1
    c["layers"][0]["mixer"]["left"]["mask"]["slide"] = 1
    c["layers"][0]["mixer"]["middle"] = {}
    HybridConfig.from_json(c)
    for key in ("twist", "slide", "middle"):
        assert key in caplog.text


@pytest.mark.parametrize("loop,want", [
    (None, [(0, -1), (1, -1), (2, -1)]),
    ((0, 1, 1), [(0, 0), (1, -1), (2, -1)]),
    ((1, 3, 2), [(0, -1), (1, 0), (2, -1), (1, 1), (2, -1)]),
    ((0, 2, 3), [(0, 0), (1, -1), (0, 1), (1, -1), (0, 2), (1, -1), (2, -1)])])
def test_order_of_runs(loop, want):
    layers = [(H.parallel(), None)] * 3
    c = H.looped(layers, loop=loop)
    assert HybridConfig.from_json(c).runs() == want
    # the oracle's own list, which marks the pass on every run of the loop
    assert [i for i, _ in O.layer_runs(c)] == [i for i, _ in want]


# ---------------------------------------------------------------- weights and caches
def test_ranks_come_from_the_weights_shapes(tmp_path):
    c = H.looped_mixed()
    full = HybridConfig.from_json(c)
    state = random_hybrid_state_dict(full, 1)
    d = HybridDecoder(HybridConfig.from_json(H.published(c)), state, device="cpu")
    assert d.cfg == full and set(d.state_dict()) == set(full.tensor_shapes())
    assert d.cfg.layers[1].mixer.right.gate_rank == 7
    assert d.cfg.layers[1].mixer.right.decay_rank == 30
    with pytest.raises(ValueError, match="shape of l1.mix.right.a2"):
        HybridDecoder(HybridConfig.from_json(H.published(c)),
                      dict(state, **{"l1.mix.right.a2": state["l1.mix.right.a2"][:, :4]}),
                      device="cpu")
    with pytest.raises(KeyError, match="missing parameters: l1.mix.right.g1"):
        HybridDecoder(HybridConfig.from_json(H.published(c)),
                      {k: v for k, v in state.items() if k != "l1.mix.right.g1"}, device="cpu")
    folder = H.model_folder(tmp_path, c, state)
    a, cfg = registry.read_config(folder)
    assert a.decoder_class is HybridDecoder and a.dtypes == (torch.bfloat16, torch.float32)
    assert cfg.layers[0].mixer.right.decay_rank is None
    model = registry.load_model(folder, device="cpu")
    assert model.decoder.cfg == full


def test_a_cache_keeps_one_chunk_per_run_of_a_layer():
    d = HybridDecoder(HybridConfig.from_json(H.looped_mixed()), device="cpu")
    cache = d.new_slot_cache(3, 80)
    assert len(cache.layers) == 6 == len(d.runs)
    rows = lambda: [t["keys"].shape[2] for t in cache.layers]
    assert rows() == [37, 80, 64, 80, 64, 80]
    assert [t["values"].shape[1] for t in cache.layers] == [2, 4, 1, 4, 1, 2]
    assert cache.layers[1]["keys"].data_ptr() != cache.layers[3]["keys"].data_ptr()
    assert cache.layers[1]["rec"].shape == (3, 3, 16, 64)
    assert cache.layers[5]["conv"].shape[1] == 1
    for t in cache.layers:
        t["keys"][2] = 3
        t["rec"][2] = 5
    cache.grow(120)
    assert rows() == [37, 100, 64, 100, 64, 120]
    assert float(cache.layers[5]["keys"][2, 1, 79, 0]) == 3
    assert float(cache.layers[5]["keys"][2, 1, 80, 0]) == 0
    cache.copy_row(2, 0, 70)
    assert float(cache.layers[0]["keys"][0, 1, 36, 0]) == 3
    assert float(cache.layers[5]["keys"][0, 0, 69, 0]) == 3
    assert float(cache.layers[4]["rec"].sum()) == 2 * 5 * cache.layers[4]["rec"][0].numel()
    assert cache.host_lens[0] == 70


# ---------------------------------------------------------------- oracle pins
def test_oracle_rotation_by_hand():
    x = torch.tensor([[[1.0, 2.0, 3.0, 4.0, 5.0]]], dtype=F64)      # pairs (0, 2) and (1, 3)
    got = O.rotate_half(x, torch.tensor([3]), 100.0, 4)[0, 0]
    a, b = 3.0, 3.0 * 100.0 ** (-0.5)
    want = [1 * math.cos(a) - 3 * math.sin(a), 2 * math.cos(b) - 4 * math.sin(b),
            3 * math.cos(a) + 1 * math.sin(a), 4 * math.cos(b) + 2 * math.sin(b), 5.0]
    assert torch.allclose(got, torch.tensor(want, dtype=F64))


def test_oracle_chunks_by_hand():
    assert O.chunk_mask(5, 2).int().tolist() == [[1, 0, 0, 0, 0], [1, 1, 0, 0, 0], [0, 0, 1, 0, 0],
                                                 [0, 0, 1, 1, 0], [0, 0, 0, 0, 1]]
    assert O.chunk_mask(3, None).int().tolist() == [[1, 0, 0], [1, 1, 0], [1, 1, 1]]


def test_oracle_grouped_attention_by_hand():
    """Two query heads of one key/value head over two positions, sizes of one."""
    one, zero = torch.ones(1, 1, dtype=F64), torch.zeros(1, dtype=F64)
    W = {"q": torch.tensor([[1.0], [2.0]], dtype=F64), "q.b": torch.tensor([0.5, 0.0], dtype=F64),
         "k": one, "k.b": zero, "v": 3 * one, "v.b": zero + 0.25,
         "g": torch.tensor([[0.0], [1.0]], dtype=F64), "o": torch.tensor([[1.0, 10.0]], dtype=F64)}
    h = torch.tensor([[1.0], [2.0]], dtype=F64)
    m = dict(heads=2, kv_heads=1, dim=1, vdim=1, scale=0.5)
    got = O.grouped_attention(h, W, "", m).view(-1)
    sig = lambda z: 1 / (1 + math.exp(-z))
    v = [3.25, 6.25]
    first = 0.5 * v[0] + 10 * sig(1.0) * v[0]
    p = [sig(0.5 * 2.5 * (2 - 1)), sig(0.5 * 4.0 * (2 - 1))]        # weight of the second key
    mix = [(1 - x) * v[0] + x * v[1] for x in p]
    second = 0.5 * mix[0] + 10 * sig(2.0) * mix[1]
    assert torch.allclose(got, torch.tensor([first, second], dtype=F64))
    got = O.grouped_attention(h, W, "", dict(m, mask=dict(size=1))).view(-1)
    assert torch.allclose(got[1], torch.tensor(0.5 * v[1] + 10 * sig(2.0) * v[1], dtype=F64))


def test_oracle_channel_decays_by_hand():
    """One head with two key channels of which one is forgotten at once: after two tokens the
    read-out of the second sees the first only through the other channel."""
    eye, zero = torch.eye(2, dtype=F64), torch.zeros(2, 2, dtype=F64)
    taps = torch.ones(2, 1, dtype=F64)
    big = 40.0      # silu(big) = big, and the unit vectors do not see the size
    W = {"q": big * torch.tensor([[0.0, 1.0], [1.0, 0.0]], dtype=F64), "k": big * eye,
         "v": torch.tensor([[30.0, 60.0]], dtype=F64), "q.conv": taps, "k.conv": taps,
         "v.conv": taps[:1], "b": torch.full((1, 2), 50.0, dtype=F64), "a1": zero[:1],
         "a2": zero[:, :1], "A_log": torch.zeros(1, dtype=F64),
         "dt_bias": torch.tensor([60.0, -60.0], dtype=F64), "g1": zero[:1], "g2": zero[:1, :1],
         "norm": torch.ones(1, dtype=F64), "o": torch.ones(1, 1, dtype=F64)}
    m = dict(heads=1, kv_heads=1, dim=2, vdim=1, conv=1)
    h = torch.tensor([[1.0, 0.0], [0.0, 1.0]], dtype=F64)
    # token 1 writes 30 under key (1, 0), which decays to nothing; token 2 asks for key (1, 0)
    got = O.channel_delta(h, W, "", m, 1e-5).view(-1)
    assert abs(float(got[0])) < 1e-6 and abs(float(got[1])) < 1e-6
    # the other way round the memory lasts: its sign is left by the norm, halved by the gate
    got = O.channel_delta(h, dict(W, dt_bias=-W["dt_bias"]), "", m, 1e-5).view(-1)
    assert torch.allclose(got[1], torch.tensor(0.5, dtype=F64), atol=1e-6)


def test_oracle_loop_terms_by_hand():
    """Mixers and feed-forwards that say nothing: only the embedding and the steps remain."""
    c = H.looped([(H.parallel(), H.dense(8))] * 3, loop=(1, 2, 3))
    W = {k: v.double() for k, v in random_hybrid_state_dict(HybridConfig.from_json(c), 3).items()}
    for k in W:
        if k.endswith(("left.out", "right.out", "mlp.down", "mlp.down.b")):
            W[k] = torch.zeros_like(W[k])
    t = torch.tensor([7, 9])
    e, s = W["embed"][t], W["loop.step"]
    logits, streams = O.forward(t, W, c, return_layers=True)
    want = [e, e + s[0], 2 * e + s[0] + s[1], 3 * e + s.sum(0), 3 * e + s.sum(0)]
    for got, x in zip(streams, want):
        assert torch.allclose(got, x)
    x = want[-1]
    x = x / torch.sqrt((x * x).mean(-1, keepdim=True) + 1e-5) * W["final.norm"]
    assert torch.allclose(logits, x @ W["embed"].T)


def test_oracle_squared_relu_and_halves_by_hand():
    W = {"up": torch.tensor([[1.0], [-1.0]]), "up.b": torch.tensor([1.0, 0.0]),
         "down": torch.tensor([[2.0, 5.0]]), "down.b": torch.tensor([0.5])}
    assert O.relu2_ff(torch.tensor([[2.0], [-3.0]]), W, "").view(-1).tolist() == [18.5, 45.5]
    c = H.looped([(H.parallel(), None)])
    W = {k: v.double() for k, v in random_hybrid_state_dict(HybridConfig.from_json(c), 4).items()}
    h, m = torch.randn(6, 72, dtype=F64), c["layers"][0]["mixer"]
    both = O.parallel(h, W, "l0.mix.", m, 1e-5)
    none = torch.zeros(72, dtype=F64)
    left = O.parallel(h, dict(W, **{"l0.mix.right.out": none}), "l0.mix.", m, 1e-5)
    right = O.parallel(h, dict(W, **{"l0.mix.left.out": none}), "l0.mix.", m, 1e-5)
    assert torch.allclose(both, left + right)
    unit = dict(W, **{"l0.mix.right.out": none, "l0.mix.left.out": none + 1})
    assert torch.allclose(O.parallel(h, unit, "l0.mix.", m, 0.0).pow(2).mean(-1),
                          torch.full((6,), 0.25, dtype=F64))


def test_oracle_is_causal():
    c = H.looped_mixed()
    W = {k: v.double() for k, v in random_hybrid_state_dict(HybridConfig.from_json(c), 2).items()}
    t = torch.randint(4, 101, (50,), generator=torch.Generator().manual_seed(1))
    assert torch.allclose(O.forward(t, W, c)[:41], O.forward(t[:41], W, c))
