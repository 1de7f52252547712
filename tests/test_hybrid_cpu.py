"""Hybrid decoders without a GPU: configuration, checkpoint reading, registry, packing, the trace
runner's bookkeeping, argument checks of the library, and hand-computed pins of the oracle."""
import ctypes
import io
import json
import math
import os
import re
import shutil
import subprocess

import pytest
import torch

from metaseq_amd import HybridConfig, OPTConfig, _capi, random_hybrid_state_dict
from metaseq_amd import registry, trace_run
from metaseq_amd.checkpoint_utils import read_safetensors
from metaseq_amd.config import DenseSpec, LatentAttentionSpec, MoESpec
from metaseq_amd.hybrid_decoder import HybridDecoder, pack_tiles
from oracle import hybrid_oracle as O
from tests import hybrid_common as H

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ---------------------------------------------------------------- configuration, registry, files
def test_config_reads_every_layer_kind():
    cfg = HybridConfig.from_json(H.mixed())
    assert cfg.vocab_size == 101 and cfg.width == 72 and cfg.norm_eps == 1e-5
    assert isinstance(cfg.layers[0].mlp, DenseSpec) and cfg.layers[2].mlp is None
    m = cfg.layers[3].mixer
    assert isinstance(m, LatentAttentionSpec) and m.kv_from == 1 and m.vdim == 16
    assert isinstance(cfg.layers[1].mlp, MoESpec)
    r = cfg.layers[1].mlp.router
    assert (r.groups, r.keep, r.top, r.scale) == (5, 2, 3, 1.5)
    assert cfg.layers[3].mlp.router.groups == 1 and cfg.layers[4].mlp.shared is None
    shapes = cfg.tensor_shapes()
    assert shapes["l1.mix.dkv.norm"] == (80,) and "l3.mix.dkv" not in shapes
    assert "l2.norm2" not in shapes and "l4.mlp.shared.sg" not in shapes
    assert shapes["l0.mix.q.conv"] == (40, 4) and shapes["l5.mix.ra"] == (2, 40, 40)


@pytest.mark.parametrize("break_it,match", [
    (lambda c: c["layers"][0].update(type="nothing"), "unknown mixer"),
    (lambda c: c["layers"][1]["mixer"].pop("kv_rank"), "kv_rank"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=0), "owns none"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=3), "owns none"),
    (lambda c: c["layers"][3]["mixer"].update(kv_rank=81), "differ in kv_rank"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), "multiple of kv_heads"),
    (lambda c: c["layers"][2]["mixer"].update(blocks=7), "multiple of blocks"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=5), "experts in"),
    (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "unknown kind"),
])
def test_bad_configurations_are_refused(break_it, match):
    c = json.loads(json.dumps(H.mixed()))
    break_it(c)
    with pytest.raises((ValueError, NotImplementedError), match=match):
        HybridConfig.from_json(c)


def test_unknown_keys_are_reported_not_fatal(caplog):
    c = json.loads(json.dumps(H.mixed()))
    c["layers"][0]["mixer"]["colour"] = 3
    with caplog.at_level("WARNING"):
        HybridConfig.from_json(c)
    assert "colour" in caplog.text


def test_safetensors_round_trip_and_model_folder(tmp_path):
    c = H.mixed()
    state = random_hybrid_state_dict(HybridConfig.from_json(c), 3)
    state["odd"] = torch.arange(5, dtype=torch.int32)
    H.write_safetensors(tmp_path / "model.safetensors", state)
    got = read_safetensors(str(tmp_path / "model.safetensors"))
    assert list(got) == list(state)
    assert all(torch.equal(got[k], state[k]) and got[k].dtype == state[k].dtype for k in state)
    (tmp_path / "config.json").write_text(json.dumps(c))
    arch, cfg = registry.read_config(str(tmp_path))
    assert arch.decoder_class is HybridDecoder and cfg.width == 72
    with pytest.raises(KeyError, match="unexpected: odd"):
        registry.load_model(str(tmp_path), device="cpu")
    with pytest.raises(ValueError, match="does not run"):
        registry.load_model(str(tmp_path), device="cpu", dtype=torch.float16)
    data = (tmp_path / "model.safetensors").read_bytes()
    (tmp_path / "short").write_bytes(data[:len(data) // 2])
    with pytest.raises(ValueError, match="does not fit"):
        read_safetensors(str(tmp_path / "short"))


def test_registry_knows_the_framework_s_models():
    assert registry.decoder_class(OPTConfig(2, 128, 2)).__name__ == "TransformerDecoder"
    assert registry.decoder_class(HybridConfig.from_json(H.mixed())) is HybridDecoder
    with pytest.raises(NotImplementedError):
        registry.decoder_class(object())
    with pytest.raises(ValueError, match="registered already"):
        registry.register("OPT", registry.ARCHITECTURES["OPT"])


def test_weights_are_checked_by_name_and_shape_and_run_on_the_gpu_only():
    cfg = HybridConfig.from_json(H.mixed())
    state = random_hybrid_state_dict(cfg, 1)
    d = HybridDecoder(cfg, state, device="cpu")
    assert set(d.state_dict()) == set(cfg.tensor_shapes())
    with pytest.raises(RuntimeError, match="GPU"):
        d.prepare_()
    with pytest.raises(ValueError, match="shape of head"):
        HybridDecoder(cfg, dict(state, head=state["head"][:5]), device="cpu")
    with pytest.raises(KeyError, match="missing parameters: l2.mix.lam"):
        HybridDecoder(cfg, {k: v for k, v in state.items() if k != "l2.mix.lam"}, device="cpu")


def test_cache_layout_keeps_what_the_layers_keep():
    d = HybridDecoder(HybridConfig.from_json(H.mixed()), device="cpu")
    cache = d.new_slot_cache(3, 50)
    assert set(cache.layers[1]) == {"latent"} and cache.layers[3] == {}
    assert cache.layers[1]["latent"].shape == (3, 50, 128)
    assert cache.layers[0]["rec"].shape == (3, 6, 32, 32) and cache.layers[0]["conv"].shape[1] == 3
    assert cache.layers[2]["rec"].dtype == torch.float32
    cache.layers[1]["latent"][2] = 7
    cache.grow(80)
    assert cache.layers[1]["latent"].shape == (3, 80, 128)
    assert float(cache.layers[1]["latent"][2, 49, 0]) == 7 and cache.capacity == 80
    cache.copy_row(2, 0, 50)
    assert float(cache.layers[1]["latent"][0, 49, 5]) == 7 and cache.host_lens[0] == 50


def test_pack_tiles_is_the_documented_layout():
    N, K = 32, 96
    w = torch.arange(N * K).view(N, K)
    p = pack_tiles(w).view(-1)
    for n, k in ((0, 0), (5, 9), (15, 31), (16, 0), (31, 95), (20, 40)):
        lane = 16 * ((k % 32) // 8) + n % 16
        assert int(p[((n // 16) * (K // 32) + k // 32) * 512 + lane * 8 + k % 8]) == n * K + k


# ---------------------------------------------------------------- trace runner
class _Echo:
    """Stands in for a decoder: the logits of a place are (slot, position, token)."""

    def __init__(self):
        self.caches, self.released = [], []

    def new_slot_cache(self, slots, capacity):
        cache = type("Cache", (), {})()
        cache.host_lens, cache.capacity = [-1] * slots, capacity
        cache.grow = lambda n: setattr(cache, "capacity", n)
        self.caches.append(cache)
        return cache

    def extend(self, cache, entries, want):
        rows = []
        for i, (slot, tokens) in enumerate(entries):
            at = max(0, cache.host_lens[slot])
            rows += [[slot, at + k, tokens[k]] for k in (want[i] if want else [])]
            cache.host_lens[slot] = at + len(tokens)
        return torch.tensor(rows, dtype=torch.float32).view(-1, 3) if want else None

    def release_slot(self, cache, slot):
        cache.host_lens[slot] = -1
        self.released.append(slot)


def test_trace_steps_continue_requests_and_give_slots_back():
    d = _Echo()
    pool = trace_run.SlotPool(d, 2, 4)
    run = lambda *entries: trace_run.run_step(d, pool, {"entries": [
        dict(id=i, tokens=t, want=w) for i, t, w in entries]}, torch)
    assert run(("a", [5, 6, 7], [2, 0])).tolist() == [[0, 2, 7], [0, 0, 5]]
    assert run(("b", [8], [])) is None
    assert run(("a", [9, 10], [1])).tolist() == [[0, 4, 10]]      # grown past its 4 positions
    assert d.caches[0].capacity == 5
    pool.release("a")
    assert run(("c", [3], [0])).tolist() == [[0, 0, 3]] and d.released == [0]
    # a third live request opens another cache; wanted rows keep the order of the entries
    got = run(("d", [1, 2], [1]), ("b", [4], [0]), ("c", [6], [0]))
    assert len(d.caches) == 2 and got.tolist() == [[0, 1, 2], [1, 1, 4], [0, 1, 6]]


def test_trace_runner_refuses_a_format_the_architecture_lacks(tmp_path, capsys):
    (tmp_path / "config.json").write_text(json.dumps(dict(
        architecture="OPT", decoder_layers=2, decoder_embed_dim=128, decoder_attention_heads=2)))
    rc = trace_run.main(["--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path)],
                        lines=io.StringIO(""))
    assert rc == 3 and "does not run" in capsys.readouterr().err


# ---------------------------------------------------------------- library boundary
def _declared(header):
    text = open(os.path.join(ROOT, "include", header)).read()
    text = re.sub(r"/\*.*?\*/", "", text, flags=re.S)
    return {m.group(1): [a for a in m.group(2).split(",") if a.strip() not in ("", "void")]
            for m in re.finditer(r"\b(msa_\w+)\s*\(([^;{]*?)\)\s*;", text, flags=re.S)}


def test_hybrid_library_exports_and_binding_match_the_header():
    if not os.path.exists(_capi.HYBRID_LIB_PATH):
        from metaseq_amd.csrc.build import build
        build(force=True, verbose=False, components=("hybrid",))
    lib = ctypes.CDLL(_capi.HYBRID_LIB_PATH)
    decls = _declared("metaseq_hybrid.h")
    assert len(decls) > 20
    for name, args in decls.items():
        assert hasattr(lib, name), name
        if name in _capi.HYBRID_SIGNATURES:
            assert len(_capi.HYBRID_SIGNATURES[name]) == len(args), name
        else:
            assert name in _capi.HYBRID_OTHER_SYMBOLS, name
    assert set(_capi.HYBRID_SIGNATURES) <= set(decls)


@pytest.mark.skipif(shutil.which("gcc") is None, reason="needs a C compiler")
def test_structures_match_the_header(tmp_path):
    pairs = {"msa_batch": _capi.Batch, "msa_group_linear_args": _capi.GroupLinearArgs,
             "msa_tail_args": _capi.TailArgs, "msa_linear_args": _capi.LinearArgs,
             "msa_delta_args": _capi.DeltaArgs, "msa_grouped_args": _capi.GroupedArgs,
             "msa_attention_layer": _capi.AttentionLayer, "msa_hybrid_layer": _capi.HybridLayer,
             "msa_hybrid_config": _capi.HybridConfigC, "msa_hybrid_state": _capi.HybridState,
             "msa_hybrid_step_args": _capi.HybridStepArgs}
    lines, want = [], []
    for c_name, cls in pairs.items():
        for field, _ in cls._fields_:
            lines.append('printf("%%zu\\n", offsetof(%s, %s));' % (c_name, field))
            want.append(getattr(cls, field).offset)
        lines.append('printf("%%zu\\n", sizeof(%s));' % c_name)
        want.append(ctypes.sizeof(cls))
    src = tmp_path / "o.c"
    src.write_text('#include <stdio.h>\n#include "metaseq_hybrid.h"\nint main(void) {\n%s\n'
                   'return 0; }\n' % "\n".join(lines))
    subprocess.run(["gcc", "-I", os.path.join(ROOT, "include"), "-o", str(tmp_path / "o"), str(src)],
                   check=True)
    out = subprocess.run([str(tmp_path / "o")], capture_output=True, text=True, check=True).stdout
    assert [int(x) for x in out.split()] == want


def test_arguments_are_checked_before_anything_is_launched():
    lib = _capi.load_hybrid()
    one = ctypes.c_void_p(4096)
    assert lib.msa_linear_bf16(one, one, one, one, 4, 40, 128, 40, -1, 0.0, 0, None) == -1
    assert b"multiple of" in lib.msa_last_error()
    assert lib.msa_linear_bf16(one, one, one, None, 4, 64, 128, 32, -1, 0.0, 0, None) == -1
    assert lib.msa_moe_route(one, 8, 4, 8, 3, 1, 2, 1.0, one, one, None, None) == -1
    assert lib.msa_moe_route(one, 8, 4, 8, 4, 1, 3, 1.0, one, one, None, None) == -1
    assert lib.msa_moe_plan(one, 64, 8, 16, one, one, one, one, one, one, 5, None) == -1
    assert lib.msa_flash_attention_bf16(one, 64, one, 128, one, 64, 0, 0, 1, 80, 4, 0, 1.0,
                                        None) == -1
    a = _capi.GroupLinearArgs()
    assert lib.msa_group_linear(ctypes.byref(a), None) == -1
    b = _capi.Batch()
    b.M = b.nseg = b.max_count = 1
    d = _capi.DeltaArgs()
    d.qkv = d.ba = d.decay_rate = d.dt_bias = d.state = d.o = 4096
    d.ld, d.ldba, d.heads, d.kv_heads, d.dim, d.dp, d.vp = 64, 8, 4, 3, 32, 32, 32
    assert lib.msa_delta_scan(ctypes.byref(d), ctypes.byref(b), None) == -1
    assert b"kv_heads=3" in lib.msa_last_error()
    g = _capi.GroupedArgs()
    g.q = g.k = g.v = g.k_cache = g.v_cache = g.out = 4096
    g.ld, g.heads, g.kv_heads, g.hd, g.vd, g.rows, g.scale, g.splits = 256, 2, 1, 64, 64, 8, 1.0, 1
    for field, bad in (("rot_dims", 3), ("rot_dims", 66), ("rows", 0), ("hd", 60), ("kv_heads", 3)):
        kept = getattr(g, field)
        setattr(g, field, bad)
        assert lib.msa_grouped_append(ctypes.byref(g), ctypes.byref(b), None) == -1, field
        setattr(g, field, kept)
    for seg0, seg1, longest in ((0, 0, 1), (0, 2, 1), (0, 1, 2), (-1, 1, 1)):
        assert lib.msa_grouped_attention(ctypes.byref(g), ctypes.byref(b), seg0, seg1, longest,
                                         None) == -1
    x = _capi.LinearArgs()
    x.x = x.W = x.y = 4096
    x.M, x.N, x.K, x.n32, x.act = 4, 64, 128, 64, 7
    assert lib.msa_linear(ctypes.byref(x), None) == -1
    cfg = _capi.HybridConfigC()
    h = ctypes.c_void_p()
    table = (_capi.HybridLayer * 1)()
    assert lib.msa_hybrid_create(ctypes.byref(cfg), table, ctypes.byref(h)) == -1


# ---------------------------------------------------------------- oracle pins
def test_oracle_convolution_by_hand():
    x = torch.tensor([[1.0], [2.0], [3.0]])
    w = torch.tensor([[10.0, 100.0]])     # previous, current
    assert O.causal_conv(x, w, torch.tensor([0.5])).view(-1).tolist() == [100.5, 210.5, 320.5]


def test_oracle_router_by_hand():
    # four groups of two; the best two groups hold the largest single experts (ids 1 and 6)
    z = torch.tensor([[0.0, 5.0, 4.0, 4.5, 3.0, 3.0, 6.0, 0.5]])
    ids, w = O.route(z, dict(top=3, scale=2.0, groups=dict(count=4, keep=2)))
    assert ids.tolist() == [[6, 1, 7]]
    s = torch.softmax(z, -1)[0]
    assert torch.allclose(w[0], 2.0 * s[[6, 1, 7]])
    ids, _ = O.route(z, dict(top=3, scale=2.0))
    assert ids.tolist() == [[6, 1, 3]]


def test_oracle_recurrences_by_hand():
    """One channel, one head: two steps of each recurrence written out."""
    one = torch.ones(1, 1, dtype=torch.float64)
    W = {"y": one, "y.b": torch.full((1,), 0.5).double(), "x": one, "x.b": torch.zeros(1).double(),
         "conv": one, "conv.b": torch.zeros(1).double(), "ra": torch.zeros(1, 1, 1).double(),
         "ra.b": torch.zeros(1, 1).double(), "ri": torch.zeros(1, 1, 1).double(),
         "ri.b": torch.zeros(1, 1).double(), "lam": torch.zeros(1).double(), "o": one}
    h = torch.tensor([[1.0], [2.0]], dtype=torch.float64)
    got = O.rglru(h, W, "", dict(width=1, blocks=1, conv=1), 1e-6).view(-1)
    a = math.exp(-8 * 0.5 * math.log(2.0))
    gelu = lambda z: 0.5 * z * (1 + math.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))
    s1 = math.sqrt(1 - a * a) * 0.5 * 1.0
    s2 = a * s1 + math.sqrt(1 - a * a) * 0.5 * 2.0
    assert torch.allclose(got, torch.tensor([s1 * gelu(1.5), s2 * gelu(2.5)], dtype=torch.float64))
    W = {"q": one, "k": one, "v": one, "g": one, "o": one, "b": 0 * one, "a": 0 * one,
         "q.conv": one, "k.conv": one, "v.conv": one, "A_log": torch.zeros(1).double(),
         "dt_bias": torch.zeros(1).double(), "norm": torch.ones(1).double()}
    m = dict(heads=1, kv_heads=1, dim=1, vdim=1, conv=1)
    got = O.delta(h, W, "", m, 0.0).view(-1)
    # the read-out is divided by its own size: only its sign times silu(gate) remains
    silu = lambda z: z / (1 + math.exp(-z))
    assert torch.allclose(got, torch.tensor([silu(1.0), silu(2.0)], dtype=torch.float64))


def test_oracle_is_causal_and_positions_matter():
    c = H.mixed()
    W = {k: v.double() for k, v in random_hybrid_state_dict(HybridConfig.from_json(c), 2).items()}
    t = torch.randint(4, 101, (12,), generator=torch.Generator().manual_seed(1))
    full = O.forward(t, W, c)
    assert torch.allclose(full[:7], O.forward(t[:7], W, c))
    same = O.forward(torch.full((2,), 9), W, c)
    assert not torch.allclose(same[0], same[1])
    pe = O.sinusoid(torch.tensor([0, 3]), 6)
    assert pe[0].tolist() == [0, 1, 0, 1, 0, 1]
    assert abs(float(pe[1, 2]) - math.sin(3 * 10000 ** (-2 / 6))) < 1e-12
