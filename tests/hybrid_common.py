"""Small hybrid configurations, their weights and comparisons with the plain oracle."""
import copy
import json

import torch

from metaseq_amd import HybridConfig, HybridDecoder, random_hybrid_state_dict
from oracle import hybrid_oracle as O

# error of the logits: root mean square over the vocabulary of the mean-free difference, over the
# root mean square of all logits: the most any row may have, and the median row
LIMIT = {torch.float32: 2e-5, torch.bfloat16: 6e-2}
MEDIAN = {torch.float32: 5e-6, torch.bfloat16: 2e-2}


def latent(heads=3, dim=24, vdim=40, kv_rank=80, q_rank=56, scale=0.3, kv_from=None):
    m = dict(heads=heads, dim=dim, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank, scale=scale)
    if kv_from is not None:
        m["kv_from"] = kv_from
    return "latent_attention", m


def rglru(width=96, blocks=3, conv=3):
    return "rglru", dict(width=width, blocks=blocks, conv=conv)


def delta(heads=6, kv_heads=2, dim=20, vdim=24, conv=4):
    return "delta", dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv)


def parallel(heads=6, kv_heads=2, dim=24, vdim=40, chunk=37, rot=(10000.0, 12), scale=0.25,
             delta_heads=4, delta_kv_heads=2, delta_dim=20, delta_vdim=28, conv=3, ranks=(18, 10)):
    """Grouped attention beside a delta rule with channel decays; ``ranks``: of the read-out gate's
    and the decays' low-rank projections."""
    left = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale)
    if rot:
        left["rot"] = dict(base=rot[0], dims=rot[1])
    if chunk:
        left["mask"] = dict(size=chunk)
    right = dict(heads=delta_heads, kv_heads=delta_kv_heads, dim=delta_dim, vdim=delta_vdim,
                 conv=conv, gate_rank=ranks[0], decay_rank=ranks[1])
    return "parallel", dict(left=left, right=right)


def dense(ff=136):
    return dict(kind="dense", ff=ff)


def moe(experts=10, top=3, scale=1.5, groups=(5, 2), ff=40, limit=1.5, shared=(72, 0.8)):
    router = dict(experts=experts, top=top, scale=scale)
    if groups:
        router["groups"] = dict(count=groups[0], keep=groups[1])
    out = dict(kind="moe", router=router, expert=dict(ff=ff, limit=limit))
    if shared:
        out["shared"] = dict(ff=shared[0], limit=shared[1])
    return out


def config(layers, width=72, vocab=101, eps=1e-5, scale=2.0):
    """A config.json dictionary; ``layers``: ((type, mixer), mlp) pairs."""
    return dict(architecture="Sinulorn", width=width, vocab=vocab, norm=dict(eps=eps),
                embedding=dict(scale=scale),
                layers=[dict(type=t, mixer=m, mlp=f) for (t, m), f in layers])


def looped(layers, loop=None, width=72, vocab=101, eps=1e-5):
    """The same for the design whose layers run in a loop; ``loop``: (start, stop, times)."""
    out = dict(architecture="Nomalorn", width=width, vocab=vocab, norm=dict(eps=eps),
               layers=[dict(type=t, mixer=m, mlp=f) for (t, m), f in layers])
    if loop:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


def looped_mixed(width=72):
    """Unequal layers, a loop over two of them, a layer without a feed-forward, a chunk shorter
    than most portions beside one longer than most sequences."""
    return looped([(parallel(), dense()),
                   (parallel(heads=4, kv_heads=4, dim=36, vdim=16, chunk=100, rot=(500.0, 36),
                             delta_heads=3, delta_kv_heads=3, delta_dim=36, delta_vdim=16, conv=4,
                             ranks=(7, 30)), None),
                   (parallel(heads=18, kv_heads=1, dim=16, vdim=20, chunk=64, rot=(1e5, 6),
                             delta_heads=6, delta_kv_heads=1, ranks=(5, 5)), dense(90)),
                   (parallel(chunk=1000, conv=2), dense(200))], loop=(1, 3, 2), width=width)


def published(cfg):
    """The configuration as a model folder has it: the ranks are left to the weights' shapes."""
    cfg = copy.deepcopy(cfg)
    for layer in cfg["layers"]:
        if layer["type"] == "parallel":
            for rank in ("gate_rank", "decay_rank"):
                layer["mixer"]["right"].pop(rank, None)
    return cfg


def mixed(dtype=torch.float32, width=72):
    """Every mechanism once, a borrowed latent, an expert layer without groups, a layer without a
    feed-forward.  With random weights some token's choice of experts is always so close that bf16
    rounding decides it (and the recurrences carry the other choice on), so in bf16 every
    expert is chosen; the choice itself is tested in fp32 and row by row."""
    pick = {} if dtype == torch.float32 else dict(experts=4, top=4, groups=(2, 2))
    flat = dict(pick, groups=None)
    return config([(delta(), dense()), (latent(), moe(**pick)), (rglru(), None),
                   (latent(heads=2, dim=36, vdim=16, q_rank=40, kv_from=1), moe(**flat)),
                   (delta(heads=4, kv_heads=4, dim=40, vdim=16, conv=2), moe(shared=None, **pick)),
                   (rglru(width=80, blocks=2, conv=5), dense(100))], width=width)


def no_specials(state):
    """Logits of the special ids 0 .. 3 are never the largest (a record ends at one)."""
    state.get("head", state["embed"])[:4] = 0


def steady(state):
    """Keys of the delta rules close to their queries.  A first token's read-out is (k . q) v, normed:
    with random weights k . q is sometimes so small that bf16 rounding decides its sign."""
    for name in [n for n in state if ".right.k" in n]:
        q = state[name.replace(".right.k", ".right.q")]
        state[name] = (0.8 * q.float() + 0.6 * state[name].float()).to(q.dtype)


def write_safetensors(path, tensors):
    names = {torch.bfloat16: "BF16", torch.float32: "F32", torch.int32: "I32"}
    header, blob = {"__metadata__": {"format": "pt"}}, b""
    for k, t in tensors.items():
        data = t.contiguous().view(torch.uint8).numpy().tobytes() if t.numel() else b""
        header[k] = dict(dtype=names[t.dtype], shape=list(t.shape),
                         data_offsets=[len(blob), len(blob) + len(data)])
        blob += data
    text = json.dumps(header).encode()
    with open(path, "wb") as f:
        f.write(len(text).to_bytes(8, "little") + text + blob)


def model_folder(path, cfg, state):
    """A model folder as the registry reads it."""
    write_safetensors(path / "model.safetensors", state)
    (path / "config.json").write_text(json.dumps(published(cfg)))
    return str(path)


class Case:
    """A model and its oracle; the oracle sees the weights the product loads (rounded to bf16)."""

    def __init__(self, cfg, seed=1, dtype=torch.float32, tweak=None, device="cuda"):
        self.json, self.dtype = cfg, dtype
        self.cfg = HybridConfig.from_json(cfg)
        self.state = random_hybrid_state_dict(self.cfg, seed)
        if tweak is not None:
            tweak(self.state)
        self.W = {k: v.double() for k, v in self.state.items()}
        self.decoder = HybridDecoder(HybridConfig.from_json(published(cfg)), self.state,
                                     device=device, dtype=dtype)
        self.cfg = self.decoder.cfg

    def tokens(self, n, seed=0):
        g = torch.Generator().manual_seed(seed)
        return torch.randint(4, self.cfg.vocab_size, (n,), generator=g)

    def want(self, tokens, layers=False):
        return O.forward(torch.as_tensor(tokens), self.W, self.json, layers)

    def run(self, tokens, portions=None, slot=0, cache=None):
        """Logits of every position, the tokens cut into ``portions`` (the last one repeats)."""
        n = len(tokens)
        cache = cache or self.decoder.new_slot_cache(slot + 1, n)
        out, at, k = [], 0, 0
        while at < n:
            step = n if portions is None else portions[min(k, len(portions) - 1)]
            piece = torch.as_tensor(tokens[at:at + step]).to(self.decoder.device)
            out.append(self.decoder.extend(cache, [(slot, piece)], want_all=True))
            at, k = at + step, k + 1
        return torch.cat(out)

    def check(self, got, want, what="", close_calls=0.0):
        """Every row within the limit, but for a share of ``close_calls`` of them."""
        got, want = got.double().cpu(), want.double().cpu()
        assert got.shape == want.shape, (what, got.shape, want.shape)
        assert torch.isfinite(got).all(), what
        d = got - want
        d = d - d.mean(dim=-1, keepdim=True)
        rows = d.pow(2).mean(dim=-1).sqrt() / want.pow(2).mean().sqrt()
        worst = float(rows.max())
        print("%s %s: worst row error %.2e at %d of %d" % (what, self.dtype, worst,
                                                           int(rows.argmax()), rows.numel()),
              flush=True)
        over = float((rows > LIMIT[self.dtype]).double().mean())
        assert over <= close_calls, (what, worst, over)
        assert float(rows.median()) <= MEDIAN[self.dtype], (what, float(rows.median()))
        return worst
