"""Hybrid decoders on gfx950: attention over a cached latent, grouped attention within chunks, gated
linear recurrent units and the gated delta rule, alone or side by side, with dense or routed
feed-forwards and layers that may run in a loop, behind the same interface as
``TransformerDecoder`` (``forward`` with a caller-owned ``incremental_state``, and the slot
interface of the serving loop).

Everything runs through one C call per step (msa_hybrid_step) over a flat batch of segments: a
prompt, a portion of a prompt (``extend``), a decode step of many rows, or a mix.  Weights are
padded and packed once for the kernels.  ``dtype`` torch.bfloat16 is the serving format; with
torch.float32 every product and activation is fp32.  There is no eager fallback.
"""
import ctypes
import uuid
from typing import Any, Dict, List, Optional, Sequence, Tuple

import torch

from . import _capi
from ._capi import check, ptr
from .config import (DenseSpec, HybridConfig, LatentAttentionSpec, ParallelSpec, RGLRUSpec,
                     SquaredReluSpec)
from .decoder_base import IncrementalDecoder, upload
from .kv_cache import HybridCache


def _up(n, m):
    return (n + m - 1) // m * m


def _k(n):
    """A reduction length as the linear layers want it: a multiple of 64, at least 128."""
    return max(128, _up(n, 64))


def _fit(n, sizes, what):
    for s in sizes:
        if n <= s:
            return s
    raise NotImplementedError("%s %d: the kernels are built for up to %d" % (what, n, sizes[-1]))


HEAD_SIZES = (32, 64, 96, 128, 192, 256)     # flash attention and delta-rule key sizes
GROUPED_SIZES = (64, 128, 192, 256)          # grouped attention on the matrix cores
LATENT_SIZES = (128, 192, 256, 384, 512)     # latent sizes of the matrix-core decode attention


def _pad(t, *shape):
    """``t`` in the leading corner of a zero tensor of ``shape``."""
    if tuple(t.shape) == shape:
        return t
    out = torch.zeros(shape, dtype=t.dtype, device=t.device)
    out[tuple(slice(0, n) for n in t.shape)] = t
    return out


def pack_tiles(w):
    """[N, K] -> the tile-packed order of the matrix-core kernels: 16 x 32 blocks along K within
    16-row tiles, lane 16 (k % 32 / 8) + n % 16 of a block owning 8 consecutive elements."""
    N, K = w.shape
    return w.view(N // 16, 16, K // 32, 4, 8).permute(0, 2, 3, 1, 4).contiguous().view(N, K)


class _LayerPlan:
    """Padded sizes of one layer and what it keeps per slot."""

    def __init__(self, spec, Dp):
        m, f = spec.mixer, spec.mlp
        if isinstance(m, LatentAttentionSpec):
            self.hd = _fit(max(m.dim, m.vdim), HEAD_SIZES, "attention head size")
            self.qp = _k(m.q_rank)
            fits = [r for r in LATENT_SIZES if r >= m.kv_rank]
            self.rp = fits[0] if fits else _k(m.kv_rank)
            own = m.kv_from is None
            self.n_in = self.qp + (self.rp if own else 0)
            self.ko = _k(m.heads * self.hd)
            self.keep = {"latent": self.rp} if own else {}
        elif isinstance(m, RGLRUSpec):
            self.bs = _up(m.width // m.blocks, 32)
            self.channels = m.blocks * self.bs
            self.n_in = 2 * self.channels
            self.ko = _k(self.channels)
            self.keep = {"conv": (m.conv - 1, self.channels), "rec": (self.channels,)}
        elif isinstance(m, ParallelSpec):
            a, d = m.left, m.right
            self.hd, self.vd = self._grouped_sizes(a)
            self.att = (a.heads + a.kv_heads) * self.hd + a.kv_heads * self.vd
            self._delta_sizes(d)
            self.lr = _k((d.gate_rank or 0) + (d.decay_rank or 0))
            self.n_in = self.att + self.qkv + self.lr + _up(a.heads + d.heads, 16)
            self.ko, self.kl = _k(d.heads * self.vp), _k(a.heads * self.vd)
            self.keep = {"keys": self.hd, "values": self.vd, "kv_heads": a.kv_heads,
                         "chunk": a.chunk, "conv": (d.conv - 1, self.qkv),
                         "rec": (d.heads, self.vp, self.dp)}
        else:
            self._delta_sizes(m)
            self.n_in = self.qkv + m.heads * self.vp + _up(2 * m.heads, 16)
            self.ko = _k(m.heads * self.vp)
            self.keep = {"conv": (m.conv - 1, self.qkv), "rec": (m.heads, self.vp, self.dp)}
        self.ff = self.ffe = self.ffs = self.n_ff = 0
        if isinstance(f, DenseSpec):
            self.ff = _k(f.ff)
            self.n_ff = 2 * self.ff
        elif isinstance(f, SquaredReluSpec):
            self.n_ff = self.ff = _k(f.ff)
        elif f is not None:
            self.ffe = _k(f.expert.ff)
            self.ffs = _k(f.shared.ff) if f.shared is not None else 0
            self.n_ff = 2 * self.ffs + _up(f.router.experts + (1 if self.ffs else 0), 16)

    def _delta_sizes(self, m):
        self.dp = _fit(m.dim, HEAD_SIZES, "delta-rule key size")
        self.vp = _up(m.vdim, 16)
        self.qkv = 2 * m.kv_heads * self.dp + m.heads * self.vp

    @staticmethod
    def _grouped_sizes(m):
        if max(m.dim, m.vdim) <= GROUPED_SIZES[-1]:
            return tuple(_fit(n, GROUPED_SIZES, "attention head size") for n in (m.dim, m.vdim))
        return _up(m.dim, 16), _up(m.vdim, 16)     # on the vector ALU


class HybridDecoder(IncrementalDecoder):
    """``forward(prev_output_tokens, incremental_state)`` returns fp32 ``(logits [B, T, V], extra)``
    with ``T = n`` for a prefill (empty ``incremental_state``; right-padded prompts allowed) and
    ``T = 1`` for a decode step over the full history, as ``TransformerDecoder`` does."""

    logits_dtype = torch.float32
    SLOT_MAX_ROWS = 256
    PORTION = 16384     # most tokens of one step; longer inputs run in portions

    def __init__(self, cfg: HybridConfig, state_dict=None, device="cuda", dtype=torch.bfloat16):
        super().__init__()
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("hybrid decoders run in bfloat16 or float32, not %s" % dtype)
        self.cfg = self.args = cfg
        self.dtype = dtype
        self.device = torch.device(device)
        self.padding_idx = cfg.padding_idx
        self.max_target_positions = cfg.max_target_positions
        self.inference = True
        self.layer_probe = None  # called as layer_probe(i, x) for every run of a layer, per step
        self.kv_cache_capacity: Optional[int] = None
        self._state_key = str(uuid.uuid4()) + ".hybrid_cache"
        self.Dp, self.Vp = _k(cfg.width), _up(cfg.vocab_size, 16)
        self._plan()
        self._raw: Optional[Dict[str, torch.Tensor]] = None
        self._handle = None
        self._weights: List[Any] = []
        self._workspace: Optional[torch.Tensor] = None
        self._select_lib = None
        self._hlib = None
        if state_dict is not None:
            self.load_state_dict(state_dict)

    def _plan(self):
        self.plans = [_LayerPlan(spec, self.Dp) for spec in self.cfg.layers]
        self.runs = self.cfg.runs()

    # ------------------------------------------------------------------ weights
    def load_state_dict(self, state_dict, strict=True, **kw):
        """Takes a checkpoint's tensors by name (``HybridConfig.tensor_shapes``)."""
        sd = {k[len("decoder."):] if k.startswith("decoder.") else k: v
              for k, v in state_dict.items()}
        cfg = self.cfg.with_shapes({k: tuple(v.shape) for k, v in sd.items()})
        shapes = cfg.tensor_shapes()
        missing = [n for n in shapes if n not in sd]
        unexpected = [n for n in sd if n not in shapes]
        if missing or (strict and unexpected):
            raise KeyError("missing parameters: %s; unexpected: %s"
                           % (", ".join(missing[:8]) or "none", ", ".join(unexpected[:8]) or "none"))
        for n, shape in shapes.items():
            if tuple(sd[n].shape) != tuple(shape):
                raise ValueError("shape of %s: expected %s, got %s" % (n, shape, tuple(sd[n].shape)))
        self._drop()
        self.cfg = self.args = cfg
        self._plan()
        self._raw = {n: sd[n].detach() for n in shapes}
        return self

    def load_tensors(self, named_tensors, **kw):
        return self.load_state_dict(dict(named_tensors))

    def state_dict(self, *args, **kwargs):
        if self._raw is None:
            raise RuntimeError("no weights are loaded")
        return dict(self._raw)

    def _drop(self):
        d = self.__dict__
        if d.get("_handle") is not None:
            d["_hlib"].msa_hybrid_destroy(d["_handle"])
        d["_handle"], d["_weights"] = None, []

    def __del__(self):
        self._drop()

    # weight transforms; every result is kept alive in self._weights and returned as a pointer
    def _hold(self, t):
        t = t.to(self.device).contiguous()
        self._weights.append(t)
        return t.data_ptr()

    def _vec(self, t, *shape):
        t = t.to(self.device).float()
        return self._hold(_pad(t, *shape) if shape else t)

    def _mat(self, w, N, K):
        """A matrix [n, k] padded to [N, K] in the step's format."""
        w = _pad(w.to(self.device), N, K)
        if self.dtype == torch.float32:
            return self._hold(w.float())
        return self._hold(pack_tiles(w.to(torch.bfloat16)))

    def _heads(self, w, heads, size, padded):
        """Rows [heads * size, k] -> [heads * padded, k]."""
        w = w.to(self.device)
        return _pad(w.view(heads, size, -1), heads, padded, w.shape[-1]).reshape(heads * padded, -1)

    def _head_columns(self, w, heads, size, padded):
        w = w.to(self.device)
        return _pad(w.view(-1, heads, size), w.shape[0], heads, padded).reshape(w.shape[0], -1)

    @staticmethod
    def _pairs(gate, up, padded):
        """(gate, up) row pairs: row 2 i is gate i, row 2 i + 1 up i."""
        k = gate.shape[1]
        return torch.stack([_pad(gate, padded, k), _pad(up, padded, k)], dim=1).view(2 * padded, k)

    def _fill_mixer(self, t, spec, plan, w):
        m, D = spec.mixer, self.cfg.width
        t.n_in, t.ko = plan.n_in, plan.ko
        if isinstance(m, LatentAttentionSpec):
            H, hd, qp, rp = m.heads, plan.hd, plan.qp, plan.rp
            t.kind, t.heads, t.hd, t.scale = _capi.MSA_MIX_LATENT, H, hd, m.scale
            t.q_rank, t.qp, t.kv_rank, t.rp = m.q_rank, qp, m.kv_rank, rp
            t.kv_from = -1 if m.kv_from is None else m.kv_from
            down = _pad(w("mix.dq").to(self.device), qp, D)
            if m.kv_from is None:
                down = torch.cat([down, _pad(w("mix.dkv").to(self.device), rp, D)])
                t.wkv_norm = self._vec(w("mix.dkv.norm"), rp)
            t.w_in = self._mat(down, plan.n_in, self.Dp)
            t.wq_norm = self._vec(w("mix.dq.norm"), qp)
            t.w_q = self._mat(self._heads(w("mix.uq"), H, m.dim, hd), H * hd, qp)
            uk = _pad(self._heads(w("mix.uk"), H, m.dim, hd), H * hd, rp)
            uv = _pad(self._heads(w("mix.uv"), H, m.vdim, hd), H * hd, rp)
            if self.dtype != torch.float32:
                t.w_kv = self._mat(torch.cat([uk, uv]), 2 * H * hd, rp)
            t.w_absorb = self._mat(uk.view(H, hd, rp).transpose(1, 2).reshape(H * rp, hd), H * rp,
                                   hd)
            t.w_v = self._mat(uv, H * hd, rp)
            t.w_out = self._mat(self._head_columns(w("mix.o"), H, m.vdim, hd), self.Dp, plan.ko)
        elif isinstance(m, RGLRUSpec):
            nb, bs, bp, C = m.blocks, m.width // m.blocks, plan.bs, plan.channels
            t.kind, t.channels, t.blocks, t.taps = _capi.MSA_MIX_RGLRU, C, nb, m.conv

            def rows(name):
                return self._heads(w(name), nb, bs, bp)

            def vec(name):
                return _pad(w(name).to(self.device).float().reshape(nb, bs), nb, bp).reshape(C)
            t.w_in = self._mat(torch.cat([rows("mix.y"), rows("mix.x")]), plan.n_in, self.Dp)
            t.y_bias, t.in_bias = self._hold(vec("mix.y.b")), self._hold(vec("mix.x.b"))
            t.conv_w = self._hold(rows("mix.conv").float().t())
            t.conv_b, t.lam = self._hold(vec("mix.conv.b")), self._hold(vec("mix.lam"))
            gates = torch.cat([_pad(w(n).to(self.device), nb, bp, bp) for n in ("mix.ra", "mix.ri")])
            t.w_gates = self._mat(gates.view(2 * nb * bp, bp), 2 * nb * bp, bp)
            t.gate_bias = self._hold(torch.cat([vec("mix.ra.b"), vec("mix.ri.b")]))
            t.w_out = self._mat(self._head_columns(w("mix.o"), nb, bs, bp), self.Dp, plan.ko)
        elif isinstance(m, ParallelSpec):
            self._fill_parallel(t, m, plan, w)
        else:
            H, Hk, dp, vp = m.heads, m.kv_heads, plan.dp, plan.vp
            t.kind, t.heads, t.kv_heads, t.taps = _capi.MSA_MIX_DELTA, H, Hk, m.conv
            t.dim, t.dp, t.vdim, t.vp = m.dim, dp, m.vdim, vp
            rows, conv = self._delta_rows(m, plan, w, "mix.")
            rows += [self._heads(w("mix.g"), H, m.vdim, vp)]
            rows += [w("mix.b").to(self.device), w("mix.a").to(self.device)]
            t.w_in = self._mat(torch.cat(rows), plan.n_in, self.Dp)
            t.conv_w = self._hold(conv)
            t.decay_rate = self._hold(torch.exp(w("mix.A_log").to(self.device).float()))
            t.dt_bias, t.o_norm = self._vec(w("mix.dt_bias")), self._vec(w("mix.norm"), vp)
            t.w_out = self._mat(self._head_columns(w("mix.o"), H, m.vdim, vp), self.Dp, plan.ko)

    def _delta_rows(self, m, plan, w, pre):
        """q, k and v rows of a delta rule and its convolution's taps [taps, channels]."""
        split = [("q", m.kv_heads, m.dim, plan.dp), ("k", m.kv_heads, m.dim, plan.dp),
                 ("v", m.heads, m.vdim, plan.vp)]
        conv = torch.cat([self._heads(w(pre + n + ".conv"), h, s, p) for n, h, s, p in split])
        return [self._heads(w(pre + n), h, s, p) for n, h, s, p in split], conv.float().t()

    def _fill_parallel(self, t, m, plan, w):
        a, d, D, Dp = m.left, m.right, self.cfg.width, self.Dp
        dev = lambda name: w("mix." + name).to(self.device)
        t.kind, at = _capi.MSA_MIX_PARALLEL, t.att
        at.heads, at.kv_heads, at.hd, at.vd = a.heads, a.kv_heads, plan.hd, plan.vd
        at.chunk, at.rot_dims, at.ko, at.scale = a.chunk or 0, a.rot_dims, plan.kl, a.scale
        i = torch.arange(a.rot_dims // 2, dtype=torch.float64)
        if a.rot_dims:
            at.inv_freq = self._hold(float(a.rot_base) ** (-2.0 * i / a.rot_dims))
        t.heads, t.kv_heads, t.taps = d.heads, d.kv_heads, d.conv
        t.dim, t.dp, t.vdim, t.vp = d.dim, plan.dp, d.vdim, plan.vp
        # the inputs of every projection of the layer's input, in one matrix
        split = [("left.q", a.heads, a.dim, plan.hd), ("left.k", a.kv_heads, a.dim, plan.hd),
                 ("left.v", a.kv_heads, a.vdim, plan.vd)]
        rows = [self._heads(dev(n), h, s, p) for n, h, s, p in split]
        column = lambda name: dev(name).float().view(-1, 1)
        bias = [self._heads(column(n + ".b"), h, s, p).view(-1) for n, h, s, p in split]
        delta, conv = self._delta_rows(d, plan, w, "mix.right.")
        low = torch.cat([dev("right.g1"), dev("right.a1")])
        rows += delta + [_pad(low, plan.lr, low.shape[1]), dev("left.g"), dev("right.b")]
        t.w_in = self._mat(torch.cat(rows), plan.n_in, Dp)
        t.in_bias, t.conv_w = self._vec(torch.cat(bias), plan.n_in), self._hold(conv)
        # gate and decays from the low-rank inputs, block-diagonal
        H, dp, vp, rg, ra = d.heads, plan.dp, plan.vp, d.gate_rank, d.decay_rank
        lr = torch.zeros(H * (vp + dp), plan.lr, dtype=dev("right.g2").dtype, device=self.device)
        lr[:H * vp, :rg] = self._heads(dev("right.g2"), H, d.vdim, vp)
        lr[H * vp:, rg:rg + ra] = self._heads(dev("right.a2"), H, d.dim, dp)
        t.lr, t.w_lr = plan.lr, self._mat(lr, H * (vp + dp), plan.lr)
        dt = self._heads(column("right.dt_bias"), H, d.dim, dp).view(-1)
        t.lr_bias = self._hold(torch.cat([torch.zeros(H * vp, device=self.device), dt]))
        rate = torch.exp(dev("right.A_log").float()).view(H, 1).expand(H, d.dim)
        t.lr_rate = self._vec(rate, H, dp)
        t.o_norm = self._vec(w("mix.right.norm"), vp)
        left = self._head_columns(dev("left.o"), a.heads, a.vdim, plan.vd)
        right = self._head_columns(dev("right.o"), H, d.vdim, vp)
        if plan.kl == plan.ko and self.dtype == torch.bfloat16:     # one product for both sides
            sides = [_pad(x, D, plan.ko) for x in (right, left)]
            t.w_out = self._mat(torch.cat(sides, dim=1), Dp, 2 * plan.ko)
        else:
            t.w_out, at.w_out = self._mat(right, Dp, plan.ko), self._mat(left, Dp, plan.kl)
        # half of each side
        at.out_norm = self._vec(0.5 * dev("left.out").float(), Dp)
        t.out_norm = self._vec(0.5 * dev("right.out").float(), Dp)

    def _fill_feed_forward(self, t, spec, plan, w):
        f, Dp = spec.mlp, self.Dp
        if f is None:
            t.ff_kind = _capi.MSA_FF_NONE
            return
        dev = lambda name: w("mlp." + name).to(self.device)
        t.n_ff_in = plan.n_ff
        if isinstance(f, DenseSpec):
            t.ff_kind, t.ff = _capi.MSA_FF_DENSE, plan.ff
            t.w_ff_in = self._mat(self._pairs(dev("gate"), dev("up"), plan.ff), plan.n_ff, Dp)
            t.w_ff_down = self._mat(dev("down"), Dp, plan.ff)
            return
        if isinstance(f, SquaredReluSpec):
            t.ff_kind, t.ff = _capi.MSA_FF_RELU2, plan.ff
            t.w_ff_in, t.w_ff_down = self._mat(dev("up"), plan.ff, Dp), self._mat(dev("down"), Dp,
                                                                                  plan.ff)
            t.ff_bias, t.ff_down_bias = self._vec(dev("up.b"), plan.ff), self._vec(dev("down.b"), Dp)
            return
        r = f.router
        t.ff_kind, t.experts, t.top = _capi.MSA_FF_MOE, r.experts, r.top
        t.n_groups, t.keep, t.router_scale = r.groups, r.keep, r.scale
        t.ff_expert, t.ff_shared, t.limit_expert = plan.ffe, plan.ffs, f.expert.limit
        rows = [dev("router")]
        if f.shared is not None:
            t.limit_shared = f.shared.limit
            rows = [self._pairs(dev("shared.gate"), dev("shared.up"), plan.ffs)] + rows \
                + [dev("shared.sg")]
            t.w_ff_down = self._mat(dev("shared.down"), Dp, plan.ffs)
        t.w_ff_in = self._mat(torch.cat(rows), plan.n_ff, Dp)
        n_in, n_dn = 2 * plan.ffe, Dp
        ins = torch.cat([_pad(self._pairs(dev("e%d.gate" % e), dev("e%d.up" % e), plan.ffe), n_in, Dp)
                         for e in range(r.experts)])
        t.w_e_in = self._mat(ins, r.experts * n_in, Dp)
        del ins
        t.w_e_down = self._mat(torch.cat([_pad(dev("e%d.down" % e), n_dn, plan.ffe)
                                          for e in range(r.experts)]),
                               r.experts * n_dn, plan.ffe)

    def prepare_(self):
        """Pads and packs the weights and creates the step handle (idempotent).  Returns the
        library of the selection and sampling kernels."""
        if self._select_lib is None:
            self._select_lib = _capi.load()
        self._prepare()
        return self._select_lib

    def _prepare(self):
        lib = self._hlib = self._hlib or _capi.load_hybrid()
        if self._handle is not None:
            return lib
        if self._raw is None:
            raise RuntimeError("no weights are loaded")
        if self.device.type != "cuda":
            raise RuntimeError("metaseq_amd: the model must live on the GPU (no CPU path exists)")
        cfg, raw, D, Dp = self.cfg, self._raw, self.cfg.width, self.Dp
        table = (_capi.HybridLayer * len(cfg.layers))()
        for i, (spec, plan) in enumerate(zip(cfg.layers, self.plans)):
            t = table[i]
            w = lambda name, pre="l%d." % i: raw[pre + name]
            self._fill_mixer(t, spec, plan, w)
            self._fill_feed_forward(t, spec, plan, w)
            for n in cfg.norm_names(spec):
                setattr(t, n, self._vec(w(n), Dp))
        c = _capi.HybridConfigC()
        c.dtype = _capi.MSA_F32 if self.dtype == torch.float32 else _capi.MSA_BF16
        c.layers, c.D, c.Dp = len(cfg.layers), D, Dp
        c.vocab, c.Vp = cfg.vocab_size, self.Vp
        c.eps, c.embed_scale = cfg.norm_eps, cfg.embed_scale
        c.embed = self._hold(_pad(raw["embed"].to(self.device).to(torch.bfloat16),
                                  cfg.vocab_size, Dp))
        if cfg.sinusoidal:
            i = torch.arange((D + 1) // 2, dtype=torch.float64)
            c.inv_freq = self._hold(10000.0 ** (-2.0 * i / D))
        c.final_norm = self._vec(raw["final.norm"], Dp)
        c.head = self._mat(raw["embed" if cfg.tied else "head"], self.Vp, Dp)
        tables = [(ctypes.c_int32 * len(self.runs))(*x) for x in zip(*self.runs)]
        c.n_runs, (c.run_layer, c.run_pass) = len(self.runs), tables
        if cfg.loop is not None:
            c.loop_step = self._vec(raw["loop.step"], cfg.loop.times, Dp)
        handle = ctypes.c_void_p()
        check(lib.msa_hybrid_create(ctypes.byref(c), table, ctypes.byref(handle)), lib)
        self._handle = handle
        return lib

    # ------------------------------------------------------------------ cache
    def max_positions(self):
        return self.max_target_positions

    def _new_cache(self, slots, capacity):
        return HybridCache([self.plans[i].keep for i, _ in self.runs], slots, capacity, self.dtype, self.device)

    def new_slot_cache(self, slots: int, capacity: int, device=None) -> HybridCache:
        """An empty cache of ``slots`` rows and ``capacity`` positions each."""
        if not 1 <= slots <= self.SLOT_MAX_ROWS:
            raise ValueError("a slot cache holds 1..%d rows" % self.SLOT_MAX_ROWS)
        if not 1 <= int(capacity) <= self.max_positions():
            raise ValueError("capacity %d outside 1..%d" % (capacity, self.max_positions()))
        return self._new_cache(slots, int(capacity))

    def _state_table(self, cache):
        key = tuple(x.data_ptr() for t in cache.layers for x in t.values())
        kept = cache.__dict__.get("_table")
        if kept is None or kept[0] != key:
            table = (_capi.HybridState * len(cache.layers))()
            for s, t in zip(table, cache.layers):
                s.latent, s.conv, s.rec = ptr(t.get("latent")), ptr(t.get("conv")), ptr(t.get("rec"))
                if "keys" in t:
                    s.keys, s.values, s.kv_rows = ptr(t["keys"]), ptr(t["values"]), t["keys"].shape[2]
            kept = cache._table = (key, table)
        return kept[1]

    # ------------------------------------------------------------------ the step
    def _step(self, cache, batch, tokens, rows=None, n_rows=0, want=True, keep=()):
        """One msa_hybrid_step.  ``rows``: int32 device tensor of the flat rows whose logits are
        wanted (None: all).  Returns fp32 logits [rows, vocab] (a view of padded rows) or None."""
        lib = self._prepare()
        a = _capi.HybridStepArgs()
        a.batch, a.tokens = batch, tokens.data_ptr()
        a.state, a.capacity = self._state_table(cache), cache.capacity
        logits = probe = None
        if want:
            n = n_rows if rows is not None else batch.M
            logits = torch.empty(n, self.Vp, dtype=torch.float32, device=self.device)
            a.rows, a.n_rows, a.logits = ptr(rows), n_rows, logits.data_ptr()
        if self.layer_probe is not None:
            probe = torch.empty(len(self.runs), batch.M, self.Dp, dtype=torch.float32,
                                device=self.device)
            a.probe = probe.data_ptr()
        need = lib.msa_hybrid_workspace_bytes(self._handle, ctypes.byref(a))
        if self._workspace is None or self._workspace.numel() < need:
            self._workspace = None
            self._workspace = torch.zeros(int(need * 1.1) + 4096, dtype=torch.uint8,
                                          device=self.device)
        a.workspace, a.workspace_bytes = self._workspace.data_ptr(), self._workspace.numel()
        check(lib.msa_hybrid_step(self._handle, ctypes.byref(a), _capi.stream_ptr()), lib)
        if probe is not None:
            for i in range(len(self.runs)):
                self.layer_probe(i, probe[i, :, :self.cfg.width])
        return None if logits is None else logits[:, :self.cfg.vocab_size]

    def _segments(self, segments: Sequence[Tuple[int, int, int]]):
        """Batch descriptor of ``segments`` ((slot, first position, tokens) each)."""
        starts, slots, pos, tok = [0], [], [], [[], [], []]
        for slot, p, n in segments:
            starts.append(starts[-1] + n)
            slots.append(slot)
            pos.append(p)
            tok[0] += [slot] * n
            tok[1] += range(p, p + n)
            tok[2] += range(n)
        M, S = starts[-1], len(slots)
        dev = upload(tok[0] + tok[1] + tok[2] + starts + slots + pos, torch.int32, self.device)
        b = _capi.Batch()
        b.M, b.nseg = M, S
        b.max_count = max(n for _, _, n in segments)
        b.key_bound = max(p + n for _, p, n in segments)
        base = dev.data_ptr()
        b.tok_slot, b.tok_pos, b.tok_off = base, base + 4 * M, base + 8 * M
        at = base + 12 * M
        b.seg_start, b.seg_slot, b.seg_pos = at, at + 4 * (S + 1), at + 4 * (2 * S + 1)
        host = [(ctypes.c_int32 * len(x))(*x) for x in (starts, slots, pos)]
        b.host_start, b.host_slot, b.host_pos = host
        return b, (dev, host)

    def extend(self, cache: HybridCache, entries, want: Optional[Sequence[Sequence[int]]] = None,
               want_all=False):
        """Runs the next tokens of several slots: ``entries`` is a list of (slot, ids), ids a
        1-D tensor or list that continues what the slot holds (an empty slot starts at
        position 0).  ``want``: per entry the offsets among its tokens whose logits are returned,
        fp32 [sum of wanted, vocab] in that order (None: no logits; ``want_all``: every token's).
        Inputs of more than PORTION tokens run in portions."""
        segments, ids = [], []
        for slot, t in entries:
            if not 0 <= slot < cache.batch:
                raise ValueError("slot %d outside 0..%d" % (slot, cache.batch - 1))
            t = t if torch.is_tensor(t) else upload(list(t), torch.long, self.device)
            if t.dim() != 1 or t.numel() == 0 or not t.is_cuda:
                raise AssertionError("tokens must be non-empty 1-D device tensors")
            pos = max(0, cache.host_lens[slot])
            if pos + t.numel() > cache.capacity:
                raise ValueError("slot %d: %d + %d positions do not fit a cache of %d"
                                 % (slot, pos, t.numel(), cache.capacity))
            segments.append((slot, pos, t.numel()))
            ids.append(t.long())
        if len({s for s, _, _ in segments}) != len(segments):
            raise ValueError("a slot is named twice")
        if want_all:
            want = [range(n) for _, _, n in segments]
        total = sum(n for _, _, n in segments)
        if total > self.PORTION:
            return self._extend_in_portions(cache, segments, ids, want)
        flat = ids[0] if len(ids) == 1 else torch.cat(ids)
        flat = flat.contiguous()
        batch, alive = self._segments(segments)
        rows, n_rows = None, 0
        if want is not None and not want_all:
            picked, at = [], 0
            for (_, _, n), w in zip(segments, want):
                if any(not 0 <= k < n for k in w):
                    raise ValueError("a wanted place lies outside the entry's tokens")
                picked += [at + k for k in w]
                at += n
            n_rows = len(picked)
            if n_rows:
                rows = upload(picked, torch.int32, self.device)
        logits = self._step(cache, batch, flat, rows, n_rows, want_all or n_rows > 0)
        del alive
        for slot, pos, n in segments:
            cache.host_lens[slot] = pos + n
            cache.lens[slot:slot + 1].fill_(pos + n)
        if want is not None and logits is None:
            logits = torch.empty(0, self.cfg.vocab_size, dtype=torch.float32, device=self.device)
        return logits

    def _extend_in_portions(self, cache, segments, ids, want):
        out = []
        for (slot, _, n), t, w in zip(segments, ids, want or [None] * len(ids)):
            places, pieces = [], []     # wanted places may come in any order
            for a in range(0, n, self.PORTION):
                b = min(n, a + self.PORTION)
                here = None if w is None else [k for k in w if a <= k < b]
                got = self.extend(cache, [(slot, t[a:b])],
                                  None if here is None else [[k - a for k in here]])
                if here:
                    places += here
                    pieces.append(got)
            if pieces:
                at = {k: j for j, k in enumerate(places)}
                out.append(torch.cat(pieces)[upload([at[k] for k in w], torch.long, self.device)])
        if want is None:
            return None
        return torch.cat(out) if out else torch.empty(
            0, self.cfg.vocab_size, dtype=torch.float32, device=self.device)

    # ------------------------------------------------------------------ decode
    def _decode(self, cache, tokens, stride, step_pos, key_bound):
        """One token for every row of ``cache`` at the positions ``step_pos`` (int32 [B] on the
        device, negative: the row sits the step out).  Returns logits [B, vocab]."""
        B = cache.batch
        fixed = cache.__dict__.get("_decode_tables")
        if fixed is None:
            r = torch.arange(B + 1, dtype=torch.int32, device=self.device)
            fixed = cache._decode_tables = (r, torch.zeros_like(r))
        r, zero = fixed
        b = _capi.Batch()
        b.M = b.nseg = B
        b.max_count, b.key_bound = 1, max(1, min(key_bound, cache.capacity))
        b.tok_slot, b.tok_pos, b.tok_off = r.data_ptr(), step_pos.data_ptr(), zero.data_ptr()
        b.seg_start, b.seg_slot, b.seg_pos = r.data_ptr(), r.data_ptr(), step_pos.data_ptr()
        if stride != 1:
            tokens = tokens.contiguous()
        return self._step(cache, b, tokens)

    def forward(self, prev_output_tokens, incremental_state: Optional[Dict[str, Any]] = None,
                features_only: bool = False, **unsupported):
        for name in ("token_embeddings", "self_attn_padding_mask"):
            if unsupported.get(name) is not None:
                raise NotImplementedError("hybrid decoders take no %s" % name)
        if features_only:
            raise NotImplementedError("hybrid decoders return logits only")
        tokens = prev_output_tokens
        if tokens.dim() != 2:
            raise AssertionError("prev_output_tokens must be [batch, tgt_len]")
        if not tokens.is_cuda:
            raise RuntimeError("metaseq_amd: tokens must live on the GPU (no CPU path exists)")
        tokens = tokens.long()
        cache = self.get_cache(incremental_state)
        if cache is None:
            logits = self._prefill(tokens, incremental_state)
        else:
            logits = self._decode_history(tokens, cache).unsqueeze(1)
        return logits, {"inner_states": []}

    def _prefill(self, tokens, incremental_state):
        B, n = tokens.shape
        pads = tokens.eq(self.padding_idx)
        counts = (n - pads.sum(dim=1)).tolist()
        trailing = torch.arange(n, device=tokens.device).unsqueeze(0) >= torch.tensor(
            counts, device=tokens.device).unsqueeze(1)
        if min(counts) < 1 or not torch.equal(pads, trailing):
            raise ValueError("hybrid decoders take right-padded prompts of at least one token")
        cap = max(int(self.kv_cache_capacity or n + 256), n)
        cache = self._new_cache(B, cap)
        logits = self.extend(cache, [(b, tokens[b, :counts[b]]) for b in range(B)], want_all=True)
        cache.length = n
        if incremental_state is not None:
            incremental_state[self._state_key] = cache
        if min(counts) == n and logits.stride(0) == self.Vp:
            return logits.unflatten(0, (B, n))
        out = torch.zeros(B, n, self.cfg.vocab_size, dtype=torch.float32, device=self.device)
        out[~pads] = logits
        return out

    def _decode_history(self, tokens, cache):
        """Decode step from the full history: the last column is the new token; a row whose new
        token is a pad sits it out."""
        lib = self._prepare()
        B, n = tokens.shape
        if n != cache.length + 1 or cache.batch != B:
            raise AssertionError("decode step expects the full history [B=%d, %d], got [%d, %d]"
                                 % (cache.batch, cache.length + 1, B, n))
        if n > self.max_positions():
            raise ValueError("sequence length %d exceeds %d positions" % (n, self.max_positions()))
        if n > cache.capacity:
            cache.grow(min(self.max_positions(), int(cache.capacity * 1.5) + 64))
        last = tokens[:, n - 1].contiguous()
        step_pos = cache.__dict__.setdefault("_step_pos", torch.empty_like(cache.lens))
        stream = _capi.stream_ptr()
        check(lib.msa_step_positions(ptr(cache.lens), ptr(last), 1, self.padding_idx, B,
                                     ptr(step_pos), stream), lib)
        logits = self._decode(cache, last, 1, step_pos, n)
        check(lib.msa_advance_active(ptr(cache.lens), ptr(step_pos), B, stream), lib)
        cache.length = n
        return logits

    def forward_select(self, prev_output_tokens, incremental_state, *, temperature, banned, stop,
                       finished, force_eos, eos, tok_out, tok_stride, score_out, score_stride,
                       logits_out=None, row_mode=None):
        """A decode step followed by the greedy selection of the next token (the outputs of
        ``TransformerDecoder.forward_select``)."""
        if not incremental_state:
            raise AssertionError("forward_select is a decode step: prefill first")
        lib = self.prepare_()
        logits = self._decode_history(prev_output_tokens.long(), self.get_cache(incremental_state))
        if logits_out is not None:
            logits_out.copy_(logits)
        self._greedy(lib, logits, temperature, banned, stop, finished, row_mode, force_eos, eos,
                     tok_out, tok_stride, score_out, score_stride)

    @staticmethod
    def _greedy(lib, logits, temperature, banned, stop, finished, row_mode, force_eos, eos, tok_out,
                tok_stride, score_out, score_stride):
        banned, stop = list(banned), list(stop)
        ba = (ctypes.c_int32 * max(1, len(banned)))(*banned)
        sa = (ctypes.c_int32 * max(1, len(stop)))(*stop)
        B, V = logits.shape
        check(lib.msa_greedy_select_f32(
            ptr(logits), logits.stride(0), B, V, float(temperature), ba, len(banned), sa, len(stop),
            ptr(finished), ptr(row_mode), int(force_eos), int(eos), ptr(tok_out), tok_stride,
            ptr(score_out), score_stride, None, _capi.stream_ptr()))

    # ------------------------------------------------------------------ slot interface
    def prefill_slot(self, cache: HybridCache, slot: int, tokens: torch.Tensor):
        """Runs the prompt ``tokens`` into slot ``slot`` from position 0 and activates it.
        Returns the logits of every prompt position, fp32 [T, V]."""
        return self.prefill_slots(cache, [slot], [tokens])[0]

    def prefill_slots(self, cache: HybridCache, slots, prompts):
        """One step for several prompts, each from position 0 of its slot; no padding.  Returns
        their logits, a list of fp32 [T_i, V]."""
        if len(slots) != len(prompts) or not prompts:
            raise AssertionError("one slot per prompt")
        for slot, t in zip(slots, prompts):
            if t.numel() >= cache.capacity:
                raise ValueError("a prompt of %d tokens leaves no room in a cache of %d positions"
                                 % (t.numel(), cache.capacity))
            if not 0 <= slot < cache.batch:
                raise ValueError("slot %d outside 0..%d" % (slot, cache.batch - 1))
            cache.host_lens[slot] = -1
        logits = self.extend(cache, list(zip(slots, prompts)), want_all=True)
        return list(logits.split([int(t.numel()) for t in prompts]))

    def release_slot(self, cache: HybridCache, slot: int):
        super().release_slot(cache, slot)
        cache.host_lens[slot] = -1

    def decode_slots(self, cache: HybridCache, last_tokens: torch.Tensor, *, temperature=1.0,
                     banned=(), stop=(), eos=2, row_mode=None, tok_out=None, score_out=None,
                     finished=None, logits_out=None, sampled=None):
        """One decode step over every active slot, with the arguments and outputs of
        ``TransformerDecoder.decode_slots`` (``logits_out``: fp32)."""
        lib = self.prepare_()
        B = cache.batch
        if last_tokens.shape != (B,) or last_tokens.dtype != torch.long:
            raise AssertionError("last_tokens must be int64 [%d]" % B)
        if max(cache.host_lens) + 1 > cache.capacity:
            raise ValueError("a slot is full (%d positions)" % cache.capacity)
        logits = self._decode(cache, last_tokens, last_tokens.stride(0), cache.lens,
                              max(cache.host_lens) + 1)
        check(self._hlib.msa_advance_active(ptr(cache.lens), ptr(cache.lens), B,
                                            _capi.stream_ptr()), self._hlib)
        cache.host_lens = [n + 1 if n >= 0 else n for n in cache.host_lens]
        if logits_out is not None:
            logits_out.copy_(logits)
        if tok_out is not None:
            self._greedy(lib, logits, temperature, banned, stop, finished, row_mode, False, eos,
                         tok_out, 1, score_out, 1)
        if sampled is not None:
            self._sample_rows(lib, logits, sampled, banned, stop, finished, eos, tok_out, score_out)
        return logits
