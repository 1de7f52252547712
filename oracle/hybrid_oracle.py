"""Plain, slow restatement of the hybrid decoder's mechanisms (test infrastructure only).

One function per mechanism, whole sequences at a time with explicit loops over positions for the
recurrences, in whatever floating dtype the weights arrive in (the tests use float32 and
float64).  Nothing here is shared with the product path: the configuration is the plain
dictionary of a config.json and the weights are a name -> tensor dictionary.
"""
import math

import torch
import torch.nn.functional as F


def rms(x, eps, w=None):
    y = x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)
    return y if w is None else y * w


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def sinusoid(positions, width, dtype=torch.float64):
    """[T, width]: columns 2i / 2i + 1 are the sine / cosine of p * 10000^(-2i / width)."""
    i = torch.arange((width + 1) // 2, dtype=torch.float64)
    ang = positions.double().unsqueeze(1) * 10000.0 ** (-2 * i / width)
    out = torch.stack([torch.sin(ang), torch.cos(ang)], dim=-1).flatten(1)[:, :width]
    return out.to(dtype)


def causal_conv(x, w, bias=None):
    """x [T, C], w [C, taps]; the last tap weighs the current position; a position in front of the
    sequence counts as 0."""
    T, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1 - j)
            if s >= 0:
                out[t] += x[s] * w[:, j]
    return out if bias is None else out + bias


def latent(h, W, pre, eps):
    """The cached latent [T, rank] of an attention layer that owns one."""
    return rms(h @ W[pre + "dkv"].T, eps, W[pre + "dkv.norm"])


def latent_attention(h, c, W, pre, m, eps):
    T, H = h.shape[0], m["heads"]
    dim, vdim = m["dim"], m["vdim"]
    cq = rms(h @ W[pre + "dq"].T, eps, W[pre + "dq.norm"])
    q = (cq @ W[pre + "uq"].T).view(T, H, dim)
    k = (c @ W[pre + "uk"].T).view(T, H, dim)
    v = (c @ W[pre + "uv"].T).view(T, H, vdim)
    out = torch.zeros(T, H, vdim, dtype=h.dtype)
    for i in range(T):
        s = torch.einsum("hd,jhd->hj", q[i], k[:i + 1]) * m["scale"]
        out[i] = torch.einsum("hj,jhd->hd", torch.softmax(s, dim=-1), v[:i + 1])
    return out.reshape(T, H * vdim) @ W[pre + "o"].T


def rglru(h, W, pre, m, eps):
    T, width, nb = h.shape[0], m["width"], m["blocks"]
    y = gelu_tanh(h @ W[pre + "y"].T + W[pre + "y.b"])
    u = causal_conv(h @ W[pre + "x"].T + W[pre + "x.b"], W[pre + "conv"], W[pre + "conv.b"])
    ub = u.view(T, nb, width // nb)
    gate = lambda n: torch.sigmoid(torch.einsum("boi,tbi->tbo", W[pre + n], ub)
                                   + W[pre + n + ".b"]).reshape(T, width)
    r, i = gate("ra"), gate("ri")
    log_a = -8.0 * r * F.softplus(W[pre + "lam"])
    a = torch.exp(log_a)
    drive = torch.sqrt(-torch.expm1(2 * log_a)) * i * u
    S, out = torch.zeros(width, dtype=h.dtype), torch.zeros(T, width, dtype=h.dtype)
    for t in range(T):
        S = a[t] * S + drive[t]
        out[t] = S
    return (out * y) @ W[pre + "o"].T


def delta(h, W, pre, m, eps):
    T, H, Hk, dim, vdim = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    conv = lambda n: F.silu(causal_conv(h @ W[pre + n].T, W[pre + n + ".conv"]))
    unit = lambda x: x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + 1e-6)
    q = unit(conv("q").view(T, Hk, dim)) * dim ** -0.5
    k = unit(conv("k").view(T, Hk, dim))
    v = conv("v").view(T, H, vdim)
    beta = torch.sigmoid(h @ W[pre + "b"].T)
    g = torch.exp(-torch.exp(W[pre + "A_log"])
                  * F.softplus(h @ W[pre + "a"].T + W[pre + "dt_bias"]))
    head = torch.arange(H) // (H // Hk)
    S = torch.zeros(H, dim, vdim, dtype=h.dtype)
    o = torch.zeros(T, H, vdim, dtype=h.dtype)
    for t in range(T):
        kt, qt = k[t, head], q[t, head]
        S = g[t].view(H, 1, 1) * S
        u = beta[t].unsqueeze(1) * (v[t] - torch.einsum("hdv,hd->hv", S, kt))
        S = S + torch.einsum("hd,hv->hdv", kt, u)
        o[t] = torch.einsum("hdv,hd->hv", S, qt)
    gate = F.silu(h @ W[pre + "g"].T).view(T, H, vdim)
    o = rms(o, eps, W[pre + "norm"]) * gate
    return o.reshape(T, H * vdim) @ W[pre + "o"].T


def rotate_half(x, positions, base, dims):
    """x [T, heads, dim]: rotates the pairs (i, i + dims / 2) of the first ``dims`` dimensions."""
    half = dims // 2
    f = float(base) ** (-2.0 * torch.arange(half, dtype=torch.float64) / max(dims, 1))
    ang = (positions.double().view(-1, 1) * f).unsqueeze(1)
    c, s = torch.cos(ang).to(x.dtype), torch.sin(ang).to(x.dtype)
    out = x.clone()
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half] = u * c - v * s
    out[..., half:dims] = v * c + u * s
    return out


def chunk_mask(T, size):
    """[T, T]: entry (i, j) says whether position i sees position j: none after it, none of another
    chunk of ``size`` positions (None: one chunk)."""
    m = torch.zeros(T, T, dtype=torch.bool)
    for i in range(T):
        first = 0 if size is None else i // size * size
        m[i, first:i + 1] = True
    return m


def grouped_attention(h, W, pre, m):
    """Rotary attention within chunks, several query heads per key/value head, each head's output
    scaled by a gate of its own."""
    T, H, G, dim, vdim = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    lin = lambda n: h @ W[pre + n].T + W[pre + n + ".b"]
    q, k, v = lin("q").view(T, H, dim), lin("k").view(T, G, dim), lin("v").view(T, G, vdim)
    if m.get("rot"):
        at = torch.arange(T)
        q = rotate_half(q, at, m["rot"]["base"], m["rot"]["dims"])
        k = rotate_half(k, at, m["rot"]["base"], m["rot"]["dims"])
    sees = chunk_mask(T, (m.get("mask") or {}).get("size"))
    gate = torch.sigmoid(h @ W[pre + "g"].T)
    out = torch.zeros(T, H, vdim, dtype=h.dtype)
    for i in range(H):
        g = i // (H // G)
        s = (q[:, i] @ k[:, g].T * m["scale"]).masked_fill(~sees, float("-inf"))
        out[:, i] = torch.softmax(s, dim=-1) @ v[:, g] * gate[:, i:i + 1]
    return out.reshape(T, H * vdim) @ W[pre + "o"].T


def channel_delta(h, W, pre, m, eps):
    """Gated delta rule with one decay per head and key channel and a low-rank sigmoid gate."""
    T, H, Hk, dim, vdim = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    conv = lambda n: F.silu(causal_conv(h @ W[pre + n].T, W[pre + n + ".conv"]))
    unit = lambda x: x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + 1e-6)
    q = unit(conv("q").view(T, Hk, dim)) * dim ** -0.5
    k = unit(conv("k").view(T, Hk, dim))
    v = conv("v").view(T, H, vdim)
    beta = torch.sigmoid(h @ W[pre + "b"].T)
    z = (h @ W[pre + "a1"].T) @ W[pre + "a2"].T + W[pre + "dt_bias"]
    decay = torch.exp(-torch.exp(W[pre + "A_log"]).view(1, H, 1) * F.softplus(z).view(T, H, dim))
    head = torch.arange(H) // (H // Hk)
    S = torch.zeros(H, dim, vdim, dtype=h.dtype)
    o = torch.zeros(T, H, vdim, dtype=h.dtype)
    for t in range(T):
        kt, qt = k[t, head], q[t, head]
        S = decay[t].unsqueeze(2) * S
        u = beta[t].unsqueeze(1) * (v[t] - torch.einsum("hdv,hd->hv", S, kt))
        S = S + torch.einsum("hd,hv->hdv", kt, u)
        o[t] = torch.einsum("hdv,hd->hv", S, qt)
    gate = torch.sigmoid((h @ W[pre + "g1"].T) @ W[pre + "g2"].T).view(T, H, vdim)
    o = rms(o, eps, W[pre + "norm"]) * gate
    return o.reshape(T, H * vdim) @ W[pre + "o"].T


def parallel(h, W, pre, m, eps):
    """Attention and delta rule side by side: the mean of their normed outputs."""
    left = grouped_attention(h, W, pre + "left.", m["left"])
    right = channel_delta(h, W, pre + "right.", m["right"], eps)
    return 0.5 * (rms(left, eps, W[pre + "left.out"]) + rms(right, eps, W[pre + "right.out"]))


def relu2_ff(h, W, pre):
    u = torch.relu(h @ W[pre + "up"].T + W[pre + "up.b"])
    return (u * u) @ W[pre + "down"].T + W[pre + "down.b"]


def layer_runs(cfg):
    """(layer, pass) in the order of execution; pass is None outside the loop."""
    loop, n = cfg.get("loop"), len(cfg["layers"])
    if not loop:
        return [(i, None) for i in range(n)]
    inner = range(loop["start"], loop["stop"])
    return ([(i, None) for i in range(loop["start"])]
            + [(i, t) for t in range(loop["times"]) for i in inner]
            + [(i, None) for i in range(loop["stop"], n)])


def dense_ff(h, W, pre):
    return (gelu_tanh(h @ W[pre + "gate"].T) * (h @ W[pre + "up"].T)) @ W[pre + "down"].T


def expert_ff(h, W, pre, limit):
    g = (h @ W[pre + "gate"].T).clamp(max=limit)
    u = (h @ W[pre + "up"].T).clamp(min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ W[pre + "down"].T


def route(z, router):
    """Logits [T, E] -> (ids [T, top], weights [T, top])."""
    s = torch.softmax(z, dim=-1)
    E = s.shape[1]
    eligible = torch.ones_like(s, dtype=torch.bool)
    groups = router.get("groups")
    if groups:
        n = groups["count"]
        best = s.view(-1, n, E // n).amax(dim=-1)
        kept = torch.zeros_like(best, dtype=torch.bool)
        kept.scatter_(1, best.topk(groups["keep"], dim=-1).indices, True)
        eligible = kept.repeat_interleave(E // n, dim=1)
    ids = s.masked_fill(~eligible, -1.0).topk(router["top"], dim=-1).indices
    return ids, s.gather(1, ids) * router["scale"]


def moe_ff(h, W, pre, mlp):
    ids, w = route(h @ W[pre + "router"].T, mlp["router"])
    out = torch.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        t, slot = (ids == e).nonzero(as_tuple=True)
        if len(t):
            y = expert_ff(h[t], W, pre + "e%d." % e, mlp["expert"]["limit"])
            out[t] += w[t, slot].unsqueeze(1) * y
    if mlp.get("shared"):
        gate = torch.sigmoid(h @ W[pre + "shared.sg"].T)
        out = out + gate * expert_ff(h, W, pre + "shared.", mlp["shared"]["limit"])
    return out


def embed(tokens, W, cfg):
    x = W["embed"][tokens] * cfg["embedding"]["scale"]
    return x + sinusoid(torch.arange(len(tokens)), cfg["width"], x.dtype)


def forward_looped(tokens, W, cfg):
    """Pre-norm layers of parallel mixers, a range of them run several times; (logits, streams)."""
    eps = cfg["norm"]["eps"]
    x = first = W["embed"][tokens]
    layers = []
    for i, t in layer_runs(cfg):
        if t is not None and i == cfg["loop"]["start"]:
            if t > 0:
                x = x + first
            x = x + W["loop.step"][t]
        pre = "l%d." % i
        layer = cfg["layers"][i]
        x = x + parallel(rms(x, eps, W[pre + "norm1"]), W, pre + "mix.", layer["mixer"], eps)
        if layer.get("mlp"):
            x = x + relu2_ff(rms(x, eps, W[pre + "norm2"]), W, pre + "mlp.")
        layers.append(x)
    return rms(x, eps, W["final.norm"]) @ W["embed"].T, layers


@torch.no_grad()
def forward(tokens, W, cfg, return_layers=False):
    """Logits [T, vocab] of one sequence (and the residual stream after every layer)."""
    W = dict(W)
    eps = cfg["norm"]["eps"]
    if cfg.get("architecture") == "Nomalorn":
        logits, layers = forward_looped(tokens, W, cfg)
        return (logits, torch.stack(layers)) if return_layers else logits
    x = embed(tokens, W, cfg)
    latents, layers = {}, []
    for i, layer in enumerate(cfg["layers"]):
        pre, m = "l%d." % i, layer["mixer"]
        h = rms(x, eps, W[pre + "norm1"])
        if layer["type"] == "latent_attention":
            j = m.get("kv_from")
            if j is None:
                latents[i] = latent(h, W, pre + "mix.", eps)
            y = latent_attention(h, latents[i if j is None else j], W, pre + "mix.", m, eps)
        else:
            y = {"rglru": rglru, "delta": delta}[layer["type"]](h, W, pre + "mix.", m, eps)
        x = x + rms(y, eps, W[pre + "norm1b"])
        mlp = layer.get("mlp")
        if mlp:
            h = rms(x, eps, W[pre + "norm2"])
            y = (dense_ff(h, W, pre + "mlp.") if mlp["kind"] == "dense"
                 else moe_ff(h, W, pre + "mlp.", mlp))
            x = x + rms(y, eps, W[pre + "norm2b"])
        layers.append(x)
    logits = rms(x, eps, W["final.norm"]) @ W["head"].T
    return (logits, torch.stack(layers)) if return_layers else logits


@torch.no_grad()
def greedy(prompt, n, W, cfg, banned=()):
    """Token-by-token continuation by full recomputation."""
    out = list(prompt)
    for _ in range(n):
        z = forward(torch.tensor(out), W, cfg)[-1].clone()
        z[list(banned)] = float("-inf")
        out.append(int(z.argmax()))
    return out
