"""Kernels of the hybrid library one by one against plain PyTorch on the CPU."""
import ctypes

import pytest
import torch

from metaseq_amd import _capi
from metaseq_amd._capi import check, ptr
from metaseq_amd.hybrid_decoder import pack_tiles
from oracle import hybrid_oracle as O

pytestmark = pytest.mark.gpu
BF16, F32 = torch.bfloat16, torch.float32


def gen(seed):
    return torch.Generator().manual_seed(seed)


def pack_rows(x):
    """[M, K] bf16 -> the packed activation layout of at most 128 rows."""
    M, K = x.shape
    MB = (M + 15) // 16 if M <= 64 else 8
    full = torch.zeros(MB * 16, K, dtype=x.dtype)
    full[:M] = x
    return full.view(MB, 16, K // 32, 4, 8).permute(2, 0, 3, 1, 4).contiguous()


def unpack_rows(p, M, K):
    MB = (M + 15) // 16 if M <= 64 else 8
    return p.view(K // 32, MB, 4, 16, 8).permute(1, 3, 0, 2, 4).reshape(MB * 16, K)[:M]


def close(got, want, tol, what):
    err = float((got.double().cpu() - want.double()).abs().max() / want.double().abs().max())
    print(what, "%.2e" % err, flush=True)
    assert err <= tol, (what, err)


def glu(kind, g, u, limit):
    if kind == _capi.MSA_GLU_GELU:
        return O.gelu_tanh(g) * u
    g, u = g.clamp(max=limit), u.clamp(-limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1)


# rows x features x reduction: every kernel of the bf16 products (packed streaming up to 128 rows,
# 128 x 128 tiles, four-wave tiles of three widths, ragged bottoms)
SHAPES = [(1, 64, 128), (5, 208, 192), (17, 96, 256), (33, 4096, 512), (64, 272, 128),
          (100, 1040, 320), (128, 512, 1024), (129, 48, 128), (200, 272, 192), (300, 1600, 256),
          (700, 4112, 256), (1024, 8192, 128), (1100, 16384, 192)]


@pytest.mark.parametrize("M,N,K", SHAPES)
def test_linear_bf16(M, N, K):
    lib = _capi.load_hybrid()
    print("linear_bf16", M, N, K, flush=True)
    g = gen(M + N)
    x = torch.randn(M, K, generator=g).to(BF16)
    w = (torch.randn(N, K, generator=g) * K ** -0.5).to(BF16)
    ref = x.double() @ w.double().T
    wp = pack_tiles(w).cuda()
    packed = M <= 128
    xd = (pack_rows(x) if packed else x).cuda()
    flags = _capi.MSA_IN_PACKED if packed else 0
    for n32 in sorted({N, N - 16, N // 2 // 16 * 16, 0}):
        y = torch.zeros(M, n32, dtype=BF16, device="cuda")
        y32 = torch.zeros(M, N - n32, dtype=F32, device="cuda")
        check(lib.msa_linear_bf16(ptr(xd), ptr(wp), ptr(y), ptr(y32), M, N, K, n32, -1, 0.0, flags,
                                  _capi.stream_ptr()), lib)
        if n32:
            close(y, ref[:, :n32], 6e-3, "bf16 columns of n32=%d" % n32)
        if n32 < N:
            close(y32, ref[:, n32:], 1e-5, "fp32 columns of n32=%d" % n32)
    for kind, n32 in ((_capi.MSA_GLU_GELU, N // 32 * 32), (_capi.MSA_GLU_CLAMPED, N // 64 * 32)):
        if n32 == 0:
            continue
        out_packed = packed and (n32 // 2) % 32 == 0
        MB = (M + 15) // 16 if M <= 64 else 8
        y = torch.zeros((MB * 16 if out_packed else M) * (n32 // 2), dtype=BF16, device="cuda")
        y32 = torch.zeros(M, N - n32, dtype=F32, device="cuda")
        check(lib.msa_linear_bf16(ptr(xd), ptr(wp), ptr(y), ptr(y32), M, N, K, n32, kind, 0.7,
                                  flags | (_capi.MSA_OUT_PACKED if out_packed else 0),
                                  _capi.stream_ptr()), lib)
        got = unpack_rows(y.cpu(), M, n32 // 2) if out_packed else y.view(M, n32 // 2)
        close(got, glu(kind, ref[:, 0:n32:2], ref[:, 1:n32:2], 0.7), 6e-3, "glu %d" % kind)
        if n32 < N:
            close(y32, ref[:, n32:], 1e-5, "fp32 columns beside glu")
    for S in {1, lib.msa_linear_bf16_splits(M, N, K, int(packed))}:
        part = torch.zeros(S, M, N, dtype=F32, device="cuda")
        check(lib.msa_linear_partial_bf16(ptr(xd), ptr(wp), ptr(part), M, N, K, S, flags,
                                          _capi.stream_ptr()), lib)
        close(part.sum(0), ref, 1e-5, "partial sums, S=%d" % S)


@pytest.mark.parametrize("M,N,K", [(1, 16, 32), (70, 80, 96), (200, 144, 128)])
def test_linear_f32(M, N, K):
    lib = _capi.load_hybrid()
    g = gen(M)
    x, w = torch.randn(M, K, generator=g), torch.randn(N, K, generator=g) * K ** -0.5
    ref = x.double() @ w.double().T
    n32 = N // 32 * 32
    if n32 == N:
        n32 -= 32
    xd, wd = x.cuda(), w.cuda()
    for kind in (-1, 0, 1):
        cols = n32 if kind < 0 else n32 // 2
        y = torch.zeros(M, cols, device="cuda")
        y32 = torch.zeros(M, N - n32, device="cuda")
        check(lib.msa_linear_f32(ptr(xd), ptr(wd), ptr(y), ptr(y32), M, N, K, n32, kind, 0.6,
                                 _capi.stream_ptr()), lib)
        if cols:
            want = ref[:, :n32] if kind < 0 else glu(kind, ref[:, 0:n32:2], ref[:, 1:n32:2], 0.6)
            close(y, want, 2e-6, "glu %d" % kind)
        close(y32, ref[:, n32:], 2e-6, "tail")


# one fp32 kernel serves every shape: the smaller ones do
@pytest.mark.parametrize("M,N,K,dtype", [s + (BF16,) for s in SHAPES] + [
    s + (F32,) for s in SHAPES if s[0] * s[1] <= 1 << 21])
def test_linear_with_bias_activation_and_decays(M, N, K, dtype):
    """Every kernel behind msa_linear: a bias, relu^2, a second output, fp32 columns as they are and
    as decays (logits far out on both sides among them)."""
    lib = _capi.load_hybrid()
    print("linear", M, N, K, dtype, flush=True)
    g = gen(M + N + K)
    x = torch.randn(M, K, generator=g).to(dtype)
    w = (torch.randn(N, K, generator=g) * K ** -0.5).to(dtype)
    bias = torch.randn(N, generator=g)
    bias[-8:-4], bias[-4:] = -16.0, 30.0
    ref = x.double() @ w.double().T + bias.double()
    packed = M <= 128 and dtype == BF16
    xd = (pack_rows(x) if packed else x).cuda()
    wd = (pack_tiles(w) if dtype == BF16 else w).cuda()
    bd = bias.cuda()
    MB = (M + 15) // 16 if M <= 64 else 8
    tol = 6e-3 if dtype == BF16 else 2e-6
    for n2, n32, act, decays in ((N, N, 1, 0), (N // 64 * 32, N // 32 * 32, 0, 0),
                                 (0, N // 32 * 32 - 32, 0, 1), (16, N - 16, 1, 1), (N - 16, N - 16, 0, 1),
                                 (0, 0, 0, 1)):
        rate = torch.rand(N - n32, generator=g) * 3
        rd = rate.cuda()
        out2_packed = packed and (n32 - n2) % 32 == 0
        y = torch.zeros(M, n2, dtype=dtype, device="cuda")
        y2 = torch.zeros((MB * 16 if out2_packed else M) * (n32 - n2), dtype=dtype, device="cuda")
        y32 = torch.zeros(M, N - n32, device="cuda")
        a = _capi.LinearArgs()
        a.dtype, a.x, a.W, a.M, a.N, a.K = int(dtype == F32), ptr(xd), ptr(wd), M, N, K
        a.n32, a.n2, a.act, a.bias = n32, n2, act, ptr(bd)
        a.decay_rate = ptr(rd) if decays and n32 < N else None
        a.flags = (_capi.MSA_IN_PACKED if packed else 0) | (_capi.MSA_OUT2_PACKED if out2_packed else 0)
        a.y, a.y32 = ptr(y) if n2 else None, ptr(y32) if n32 < N else None
        if n2 < n32:
            a.y2 = ptr(y2)
        check(lib.msa_linear(ctypes.byref(a), _capi.stream_ptr()), lib)
        want = torch.relu(ref) ** 2 if act else ref
        what = "n2=%d n32=%d act=%d" % (n2, n32, act)
        if n2:
            close(y, want[:, :n2], tol, what)
        if n2 < n32:
            got = unpack_rows(y2.cpu(), M, n32 - n2) if out2_packed else y2.view(M, n32 - n2)
            close(got, want[:, n2:n32], tol, "second output, " + what)
        if n32 < N:
            z = ref[:, n32:]
            if decays:
                z = torch.exp(-rate.double() * torch.nn.functional.softplus(z))
            close(y32, z, 1e-5 if dtype == BF16 else 3e-6, "fp32 columns, " + what)
            if decays:   # next to 1 the distance from 1 counts
                slow = z > 0.999
                off = ((1 - y32.cpu().double()) - (1 - z)).abs()[slow]
                assert off.numel() == 0 or float(off.max()) < 3e-7, what


@pytest.mark.parametrize("dtype", [BF16, F32], ids=["bf16", "f32"])
@pytest.mark.parametrize("M,D", [(1, 72), (5, 4096), (40, 1000), (130, 2100), (1100, 300),
                                 (1030, 5000), (3, 9000)])
def test_tail_of_two_sides_with_loop_terms(M, D, dtype):
    """Both sides' sums and norms, a bias, what a loop adds, the probe and the next norm."""
    lib = _capi.load_hybrid()
    g = gen(M + D)
    Dp, eps = (D + 63) // 64 * 64, 1e-3

    def wide(*shape):
        t = torch.zeros(*shape, Dp)
        t[..., :D] = torch.randn(*shape, D, generator=g)
        return t
    for S, S2, two, extra in ((1, 1, True, True), (3, 5, True, False), (2, 0, False, True)):
        x, part, part2 = wide(M), wide(S, M), wide(max(1, S2), M)
        bias, w, w2, add, step, nxt = wide(), wide(), wide(), wide(M), wide(), wide()
        b = part.double().sum(0) + (bias.double() if extra else 0)
        want = x.double()
        want = want + (O.rms(b[:, :D], eps, w[:D].double()) if two else b[:, :D]) \
            if Dp == D else want.clone()
        if Dp != D:
            want[:, :D] += O.rms(b[:, :D], eps, w[:D].double()) if two else b[:, :D]
        if two:
            want[:, :D] += O.rms(part2.double().sum(0)[:, :D], eps, w2[:D].double())
        probe = want.clone()
        if extra:
            want = want + add.double() + step.double()
        h = O.rms(want[:, :D], eps, nxt[:D].double())
        dev = [t.cuda() for t in (x, part, part2, bias, w, w2, add, step, nxt)]
        hd = torch.zeros(M, Dp, dtype=dtype, device="cuda")
        pd = torch.zeros(M, Dp, device="cuda")
        a = _capi.TailArgs()
        a.dtype, a.M, a.D, a.Dp, a.S, a.eps = int(dtype == F32), M, D, Dp, S, eps
        a.x, a.part, a.h, a.w_next, a.probe = ptr(dev[0]), ptr(dev[1]), ptr(hd), ptr(dev[8]), ptr(pd)
        if two:
            a.part2, a.S2, a.w_post, a.w_post2 = ptr(dev[2]), S2, ptr(dev[4]), ptr(dev[5])
        if extra:
            a.bias, a.add, a.step = ptr(dev[3]), ptr(dev[6]), ptr(dev[7])
        check(lib.msa_residual_rmsnorm_tail(ctypes.byref(a), _capi.stream_ptr()), lib)
        close(dev[0], want, 2e-6, "stream")
        close(pd, probe, 2e-6, "probe")
        close(hd[:, :D], h, 6e-3 if dtype == BF16 else 3e-6, "normed")


def _grouped(lib, dtype, heads, kv_heads, hd, vd, chunk, rot, segments, capacity, seed, fused=None):
    """One step of grouped attention over ``segments`` ((slot, first position, tokens)) through the
    three calls; returns its outputs and the caches with what they should be."""
    g = gen(seed)
    M = sum(n for _, _, n in segments)
    slots = 1 + max(s for s, _, _ in segments)
    rows = min(capacity, chunk) if chunk else capacity
    ld = (heads + kv_heads) * hd + kv_heads * vd + 16
    x = torch.randn(M, ld, generator=g).to(dtype)
    kc = torch.randn(slots, kv_heads, rows, hd, generator=g).to(dtype)
    vc = torch.randn(slots, kv_heads, rows, vd, generator=g).to(dtype)
    gate = torch.randn(M, heads + 3, generator=g)
    inv = 100.0 ** (-2.0 * torch.arange(rot // 2, dtype=torch.float64) / max(1, rot))
    scale = 1.5 * hd ** -0.5
    want, kw, vw = torch.zeros(M, heads, vd, dtype=torch.float64), kc.clone(), vc.clone()
    at = 0
    for slot, pos, n in segments:
        if pos >= 0:
            own = x[at:at + n].double()
            q = own[:, :heads * hd].view(n, heads, hd)
            k = own[:, heads * hd:(heads + kv_heads) * hd].view(n, kv_heads, hd)
            v = own[:, (heads + kv_heads) * hd:-16].view(n, kv_heads, vd)
            p = torch.arange(pos, pos + n)
            if rot:
                q, k = (O.rotate_half(t, p, 100.0, rot).to(dtype).double() for t in (q, k))
            c0 = pos // chunk * chunk if chunk else 0
            keys = torch.cat([kc[slot, :, :pos - c0].double().transpose(0, 1), k])
            vals = torch.cat([vc[slot, :, :pos - c0].double().transpose(0, 1), v])
            where = torch.arange(c0, pos + n)
            for h in range(heads):
                j = h // (heads // kv_heads)
                s = q[:, h] @ keys[:, j].T * scale
                first = p // chunk * chunk if chunk else torch.zeros_like(p)
                sees = (where <= p[:, None]) & (where >= first[:, None])
                s = s.masked_fill(~sees, float("-inf"))
                want[at:at + n, h] = torch.softmax(s, -1) @ vals[:, j] * torch.sigmoid(
                    gate[at:at + n, h:h + 1].double())
            last = (pos + n - 1) // chunk * chunk if chunk else 0
            for i in range(max(0, last - pos), n):
                kw[slot, :, pos + i - last] = k[i].to(dtype)
                vw[slot, :, pos + i - last] = v[i].to(dtype)
        at += n
    b, alive = _batch(segments, M)
    b.key_bound = max(max(p + n for _, p, n in segments), 1)
    xd, kd, vd_, gd, fd = x.cuda(), kc.cuda(), vc.cuda(), gate.cuda(), inv.cuda()
    out = torch.full((M, heads * vd), 7.0, dtype=dtype, device="cuda")
    a = _capi.GroupedArgs()
    a.dtype, a.heads, a.kv_heads, a.hd, a.vd = int(dtype == F32), heads, kv_heads, hd, vd
    a.chunk, a.rot_dims, a.rows, a.scale = chunk, rot, rows, scale
    a.inv_freq = ptr(fd) if rot else None
    es = x.element_size()
    a.q, a.k = xd.data_ptr(), xd.data_ptr() + heads * hd * es
    a.v, a.ld = a.k + kv_heads * hd * es, ld
    a.k_cache, a.v_cache, a.gate, a.ld_gate = ptr(kd), ptr(vd_), ptr(gd), heads + 3
    a.out, a.ldo = ptr(out), heads * vd
    a.fused = lib.msa_grouped_fuses(ctypes.byref(a), ctypes.byref(b)) if fused is None else fused
    part = torch.zeros(M * heads * 64 * (vd + 4), device="cuda")
    a.partial, s = ptr(part), _capi.stream_ptr()
    ref = (ctypes.byref(a), ctypes.byref(b))
    if not a.fused:
        check(lib.msa_grouped_rotate(*ref, s), lib)
    seg = 0
    counts = [n for _, _, n in segments]
    while seg < len(counts):
        end = seg + 1
        while end < len(counts) and (counts[end] == 1) == (counts[seg] == 1):
            end += 1
        a.splits = 1
        if counts[seg] == 1:
            a.splits = lib.msa_grouped_attention_splits(ctypes.byref(a), end - seg, b.key_bound)
        check(lib.msa_grouped_attention(*ref, seg, end, max(counts[seg:end]), s), lib)
        seg = end
    if not a.fused:
        check(lib.msa_grouped_append(*ref, s), lib)
    tol = 2e-5 if dtype == F32 else 1.5e-2
    on = torch.cat([torch.full((n,), p >= 0) for _, p, n in segments])
    close(out.view(M, heads, vd)[on.cuda()], want[on], tol, "outputs, splits=%d" % a.splits)
    # rotated keys in another order of operations: the last bit may differ
    close(kd, kw, 1e-6 if dtype == F32 else 8e-3, "keys kept")
    assert torch.equal(vd_.cpu(), vw), "values kept"


GROUPED = [(4, 2, 64, 64, 40), (8, 8, 128, 128, 128), (34, 2, 64, 128, 10), (3, 1, 192, 64, 0),
           (4, 1, 256, 256, 64), (2, 2, 128, 192, 126), (5, 5, 192, 256, 34), (16, 8, 256, 64, 2),
           (17, 1, 64, 192, 64), (3, 3, 80, 272, 16), (8, 8, 64, 256, 62), (2, 1, 128, 64, 0)]


@pytest.mark.parametrize("dtype", [BF16, F32], ids=["bf16", "f32"])
@pytest.mark.parametrize("heads,kv_heads,hd,vd,rot", GROUPED)
def test_grouped_attention(heads, kv_heads, hd, vd, rot, dtype):
    """Decode steps (fused and not, with and without splits), portions over several chunks, mixed
    batches with inactive segments, with and without chunks."""
    lib = _capi.load_hybrid()
    size = (heads, kv_heads, hd, vd)
    print("grouped", size, rot, flush=True)
    decode = [(2, 700, 1), (0, 0, 1), (1, -1, 1), (4, 255, 1), (3, 129, 1), (5, 511, 1)]
    mix = [(1, 250, 1), (0, 90, 70), (2, 5, 1), (3, -1, 1), (4, 0, 150), (5, 127, 2), (6, -1, 3),
           (7, 64, 64)]
    for chunk in (0, 100, 128, 1000):
        _grouped(lib, dtype, *size, chunk, rot, decode, 800, heads)
        _grouped(lib, dtype, *size, chunk, rot, decode, 800, heads, fused=0)
        _grouped(lib, dtype, *size, chunk, rot, mix, 300, heads + 1)
    _grouped(lib, dtype, *size, 7, rot, [(0, 3, 40), (1, 6, 1), (2, 0, 7), (3, 13, 2)], 300, hd)
    _grouped(lib, dtype, *size, 0, rot, [(0, 1500, 1)], 1600, hd)          # splits


@pytest.mark.parametrize("dtype", [BF16, F32], ids=["bf16", "f32"])
@pytest.mark.parametrize("M", [1, 16, 20, 64, 150])
def test_group_linear_dense(M, dtype):
    """Per-group columns (a head, a diagonal block), also with the groups' inputs shared."""
    lib = _capi.load_hybrid()
    for G, N, K, share in ((3, 48, 64, 0), (6, 160, 32, 3), (1, 272, 128, 0)):
        g = gen(M + G)
        xg = share or G
        x = torch.randn(M, xg * K, generator=g).to(dtype)
        w = (torch.randn(G, N, K, generator=g) * K ** -0.5).to(dtype)
        ref = torch.stack([x[:, (i % xg) * K:(i % xg + 1) * K].double() @ w[i].double().T
                           for i in range(G)], dim=1).view(M, G * N)
        wd = (pack_tiles(w.view(G * N, K)) if dtype == BF16 else w.view(G * N, K)).cuda()
        xd = x.cuda()
        for y_f32 in (0, 1):
            y = torch.zeros(M, G * N, dtype=F32 if y_f32 else dtype, device="cuda")
            a = _capi.GroupLinearArgs()
            a.dtype, a.glu = (0 if dtype == BF16 else 1), -1
            a.x, a.ldx, a.x_group, a.x_groups = ptr(xd), xg * K, K, share
            a.W, a.y, a.ldy, a.y_group, a.y_f32 = ptr(wd), ptr(y), G * N, N, y_f32
            a.N, a.K, a.groups, a.M = N, K, G, M
            check(lib.msa_group_linear(ctypes.byref(a), _capi.stream_ptr()), lib)
            tol = 2e-6 if dtype == F32 else (1e-5 if y_f32 else 6e-3)
            close(y, ref, tol, "groups %s" % ((G, N, K, share),))


@pytest.mark.parametrize("E,groups,keep,top", [(1, 1, 1, 1), (12, 1, 1, 5), (12, 4, 2, 3),
                                               (96, 8, 3, 10), (512, 16, 16, 8), (300, 100, 1, 3)])
def test_route_and_plan(E, groups, keep, top):
    lib = _capi.load_hybrid()
    M = 77
    z = torch.randn(M, E + 5, generator=gen(E)) * 2
    want_ids, want_w = O.route(z[:, :E].double(), dict(
        top=top, scale=1.7, groups=dict(count=groups, keep=keep)))
    zd = z.cuda()
    ids = torch.zeros(M, top, dtype=torch.int32, device="cuda")
    w = torch.zeros(M, top, device="cuda")
    sg = torch.zeros(M, device="cuda")
    check(lib.msa_moe_route(ptr(zd), E + 5, M, E, groups, keep, top, 1.7, ptr(ids), ptr(w), ptr(sg),
                            _capi.stream_ptr()), lib)
    assert torch.equal(ids.cpu().long(), want_ids)
    close(w, want_w, 1e-5, "weights")
    close(sg, torch.sigmoid(z[:, E].double()), 1e-6, "shared gate")
    P = M * top
    for rows in (16, 64):
        n_max = P // rows + min(E, P)
        perm, inv = (torch.full((P,), -1, dtype=torch.int32, device="cuda") for _ in range(2))
        end = torch.zeros(E, dtype=torch.int32, device="cuda")
        tg, tr = (torch.full((n_max,), -1, dtype=torch.int32, device="cuda") for _ in range(2))
        n = torch.zeros(1, dtype=torch.int32, device="cuda")
        check(lib.msa_moe_plan(ptr(ids), P, E, rows, ptr(perm), ptr(inv), ptr(end), ptr(tg), ptr(tr),
                               ptr(n), n_max, _capi.stream_ptr()), lib)
        flat = ids.cpu().view(-1).long()
        order = torch.sort(flat, stable=True).indices
        assert torch.equal(perm.cpu().long(), order)
        assert torch.equal(inv.cpu().long()[order], torch.arange(P))
        counts = torch.bincount(flat, minlength=E)
        assert torch.equal(end.cpu().long(), counts.cumsum(0))
        tiles = [(e, int(counts[:e].sum()) + r) for e in range(E)
                 for r in range(0, int(counts[e]), rows)]
        assert int(n) == len(tiles)
        assert list(zip(tg.cpu().tolist(), tr.cpu().tolist()))[:len(tiles)] == tiles


@pytest.mark.parametrize("hd", [32, 64, 96, 128, 192, 256])
@pytest.mark.parametrize("T,pos0", [(1, 0), (17, 3), (64, 64), (130, 0), (33, 400), (300, 100)])
def test_flash_attention(hd, T, pos0):
    lib = _capi.load_hybrid()
    heads, S = 3, T + pos0
    g = gen(hd + T)
    q = torch.randn(T, heads * hd, generator=g).to(BF16)
    kv = torch.randn(S, 2 * heads * hd, generator=g).to(BF16)
    scale = 1.5 * hd ** -0.5
    k, v = (t.double().view(S, heads, hd) for t in kv.split(heads * hd, dim=1))
    s = torch.einsum("thd,shd->hts", q.double().view(T, heads, hd), k) * scale
    mask = torch.arange(S).view(1, S) > pos0 + torch.arange(T).view(T, 1)
    p = torch.softmax(s.masked_fill(mask, float("-inf")), dim=-1)
    ref = torch.einsum("hts,shd->thd", p, v).reshape(T, heads * hd)
    out = torch.zeros(T, heads * hd, dtype=BF16, device="cuda")
    qd, kvd = q.cuda(), kv.cuda()
    check(lib.msa_flash_attention_bf16(ptr(qd), heads * hd, ptr(kvd), 2 * heads * hd, ptr(out),
                                       heads * hd, 0, 0, heads, hd, T, pos0, scale,
                                       _capi.stream_ptr()), lib)
    close(out, ref, 1e-2, "flash %d" % hd)


@pytest.mark.parametrize("dtype", [BF16, F32], ids=["bf16", "f32"])
@pytest.mark.parametrize("rp", [128, 192, 256, 384, 512, 640])
def test_latent_attention(rp, dtype):
    """Rows of several slots at their own positions, an inactive row, and one to eight splits."""
    lib = _capi.load_hybrid()
    heads, cap, slots = 19, 700, 3
    g = gen(rp)
    pos = [0, 31, 32, 127, 128, 129, 300, 640, 699, -1]
    slot = [i % slots for i in range(len(pos))]
    M = len(pos)
    c = torch.randn(slots, cap, rp, generator=g).to(dtype)
    q = torch.randn(M, heads, rp, generator=g).to(dtype)
    scale = 1.5 * rp ** -0.5
    ref = torch.zeros(M, heads, rp, dtype=torch.float64)
    for m in range(M):
        if pos[m] >= 0:
            rows = c[slot[m], :pos[m] + 1].double()
            ref[m] = torch.softmax(q[m].double() @ rows.T * scale, dim=-1) @ rows
    cd, qd = c.cuda(), q.cuda()
    ts = torch.tensor(slot, dtype=torch.int32, device="cuda")
    tp = torch.tensor(pos, dtype=torch.int32, device="cuda")
    for splits in (1, 2, 8):
        out = torch.full((M, heads, rp), 9.0, dtype=dtype, device="cuda")
        part = torch.zeros(M, heads, splits, rp + 4, device="cuda")
        check(lib.msa_latent_attention(0 if dtype == BF16 else 1, ptr(qd), ptr(cd), cap, heads, rp,
                                       scale, ptr(out), ptr(part), splits, ptr(ts), ptr(tp), M,
                                       _capi.stream_ptr()), lib)
        close(out, ref, 1e-2 if dtype == BF16 else 1e-5, "latent %d, %d splits" % (rp, splits))


def _batch(segments, M):
    """A msa_batch of (slot, first position, tokens) segments with its tensors."""
    start, slot, pos = [0], [], []
    tok = [[], [], []]
    for s, p, n in segments:
        start.append(start[-1] + n)
        slot.append(s)
        pos.append(p)
        tok[0] += [s] * n
        tok[1] += [p + i if p >= 0 else -1 for i in range(n)]
        tok[2] += range(n)
    dev = [torch.tensor(x, dtype=torch.int32, device="cuda") for x in tok + [start, slot, pos]]
    b = _capi.Batch()
    b.M, b.nseg, b.max_count = M, len(slot), max(n for _, _, n in segments)
    (b.tok_slot, b.tok_pos, b.tok_off, b.seg_start, b.seg_slot, b.seg_pos) = map(ptr, dev)
    host = [(ctypes.c_int32 * len(x))(*x) for x in (start, slot, pos)]
    b.host_start, b.host_slot, b.host_pos = host
    return b, (dev, host)


@pytest.mark.parametrize("heads,kv_heads,dim,dp,vp,counts", [
    (4, 2, 30, 32, 48, (5, 1, 40)), (3, 3, 128, 128, 64, (17, 16)), (2, 1, 250, 256, 32, (33,)),
    (32, 8, 64, 64, 64, (9, 2, 1, 30, 16, 17, 3, 4)),      # eight lanes per column
    (64, 64, 128, 128, 32, (7, 20, 1, 2, 1, 1, 1, 1)), (32, 16, 96, 96, 64, (5,) * 8),
    (6, 3, 90, 96, 80, (1, 1, 1)), (3, 1, 128, 128, 208, (1,) * 5)])
@pytest.mark.parametrize("channels", [False, True], ids=["head decays", "channel decays"])
@pytest.mark.parametrize("dtype", [BF16, F32], ids=["bf16", "f32"])
def test_delta_scan(heads, kv_heads, dim, dp, vp, counts, dtype, channels):
    """Several segments, one of them continuing its slot's state and (with three or more) one
    inactive; outputs and the states left behind.  Segments of one token each also through the
    one-launch step."""
    lib = _capi.load_hybrid()
    print("delta_scan", heads, kv_heads, dim, dp, vp, counts, channels, flush=True)
    g = gen(heads + dp)
    M, slots = sum(counts), len(counts) + 1
    C = 2 * kv_heads * dp + heads * vp
    qkv = torch.randn(M, C, generator=g)
    qkv[:, :2 * kv_heads * dp].view(M, 2 * kv_heads, dp)[:, :, dim:] = 0
    qkv = qkv.to(dtype)
    ba = torch.randn(M, 2 * heads + 3, generator=g)
    rate, dtb = torch.rand(heads, generator=g) * 0.3, torch.randn(heads, generator=g)
    decays = torch.rand(M, heads, dp, generator=g) ** 0.25
    state = torch.randn(slots, heads, vp, dp, generator=g)
    state[..., dim:] = 0
    segs = [(slots - 1 - i, 0 if i else 12, n) for i, n in enumerate(counts)]
    if len(counts) > 2:
        segs[1] = (segs[1][0], -1, segs[1][2])
    want, S = torch.zeros(M, heads, vp, dtype=torch.float64), state.double().clone()
    x = qkv.double()
    unit = lambda t: t / torch.sqrt((t * t).sum(-1, keepdim=True) + 1e-6)
    at = 0
    for slot, pos, n in segs:
        if pos >= 0:
            s = S[slot] if pos > 0 else torch.zeros_like(S[slot])       # [heads, vp, dp]
            for m in range(at, at + n):
                q = unit(x[m, :kv_heads * dp].view(kv_heads, dp)) * dim ** -0.5
                k = unit(x[m, kv_heads * dp:2 * kv_heads * dp].view(kv_heads, dp))
                q, k = (t.repeat_interleave(heads // kv_heads, 0) for t in (q, k))
                v = x[m, 2 * kv_heads * dp:].view(heads, vp)
                z = ba[m].double()
                beta = torch.sigmoid(z[:heads])
                decay = torch.exp(-rate.double() * torch.nn.functional.softplus(
                    z[heads:2 * heads] + dtb.double()))
                s = s * (decays[m].double().unsqueeze(1) if channels else decay.view(-1, 1, 1))
                u = beta.view(-1, 1) * (v - torch.einsum("hvd,hd->hv", s, k))
                s = s + u.unsqueeze(2) * k.unsqueeze(1)
                want[m] = torch.einsum("hvd,hd->hv", s, q)
            S[slot] = s
        at += n
    b, alive = _batch(segs, M)
    qd, bd, rd, td, sd, dd = (t.cuda() for t in (qkv, ba, rate, dtb, state, decays))
    o = torch.full((M, heads * vp), 7.0, device="cuda")
    a = _capi.DeltaArgs()
    a.dtype, a.heads, a.kv_heads, a.dim, a.dp, a.vp = int(dtype == F32), heads, kv_heads, dim, dp, vp
    a.qkv, a.ld, a.ba, a.ldba, a.state, a.o = ptr(qd), C, ptr(bd), 2 * heads + 3, ptr(sd), ptr(o)
    if channels:
        a.decay = ptr(dd)
    else:
        a.decay_rate, a.dt_bias = ptr(rd), ptr(td)
    if b.max_count == 1:
        step = state.cuda()
        out = torch.zeros(M, heads * vp, dtype=dtype, device="cuda")
        gate, w = torch.randn(M, heads * vp, generator=g).to(dtype), torch.randn(vp, generator=g)
        gd, wd = gate.cuda(), w.cuda()
        a.state, a.vdim, a.gate, a.ld_gate, a.w = ptr(step), vp, ptr(gd), heads * vp, ptr(wd)
        a.out, a.ld_out, a.eps = ptr(out), heads * vp, 1e-5
        for act, f in ((_capi.MSA_GATE_SILU, torch.nn.functional.silu),
                       (_capi.MSA_GATE_SIGMOID, torch.sigmoid)):
            step.copy_(state)
            a.gate_act = act
            check(lib.msa_delta_step(ctypes.byref(a), ctypes.byref(b), _capi.stream_ptr()), lib)
            normed = O.rms(want, 1e-5, w.double()) * f(gate.double()).view(M, heads, vp)
            on = [m for m in range(M) if segs[m][1] >= 0]
            close(out.view(M, heads, vp)[on], normed[on], 2e-5 if dtype == F32 else 6e-3, "step")
            close(step, S, 2e-5, "states of the step")
        a.state = ptr(sd)
    check(lib.msa_delta_scan(ctypes.byref(a), ctypes.byref(b), _capi.stream_ptr()), lib)
    close(o.view(M, heads, vp), want, 2e-5, "outputs")
    close(sd, S, 2e-5, "states")
    del alive


def test_selection_over_fp32_logits():
    """The fp32 forms of selection, scoring and sampling agree with plain PyTorch, at row strides
    and vocabulary sizes that are no multiple of 8."""
    lib = _capi.load()
    for V, ld in ((101, 112), (1000, 1000), (50001, 50016)):
        z = torch.randn(5, ld, generator=gen(V)).cuda() * 3
        lp = torch.log_softmax(z[:, :V].double(), dim=-1)
        tok = torch.zeros(5, dtype=torch.long, device="cuda")
        score = torch.zeros(5, device="cuda")
        ban = (ctypes.c_int32 * 1)(1)
        none = (ctypes.c_int32 * 1)()
        check(lib.msa_greedy_select_f32(ptr(z), ld, 5, V, 1.0, ban, 1, none, 0, None, None, 0, 2,
                                        ptr(tok), 1, ptr(score), 1, None, _capi.stream_ptr()))
        masked = lp.clone()
        masked[:, 1] = float("-inf")
        assert torch.equal(tok, masked.argmax(dim=-1))
        close(score, masked.max(dim=-1).values.cpu(), 1e-5, "score")
        target = torch.randint(0, V, (5,), generator=gen(1)).cuda()
        got = torch.zeros(5, device="cuda")
        check(lib.msa_target_logprob_f32(ptr(z), ld, 5, V, 1.0, ptr(target), ptr(got),
                                         _capi.stream_ptr()))
        close(got, lp.gather(1, target.view(-1, 1)).view(-1).cpu(), 1e-5, "target")
        rows = torch.zeros(5, V, device="cuda")
        check(lib.msa_log_softmax_f32(ptr(z), 0, ld, 1, 5, V, 1.0, ptr(rows), 0, V,
                                      _capi.stream_ptr()))
        close(rows, lp.cpu(), 1e-5, "log-softmax")
        noise = torch.empty(5, V, device="cuda").exponential_()
        check(lib.msa_sample_topp_f32(ptr(z), ld, 5, V, 1.0, None, ban, 1, none, 0, None, None, 0, 2,
                                      None, 0.999999, ptr(noise), None, None, 0.0, 0.0, 0.0, 0.0,
                                      None, None, 0, ptr(tok), 1, ptr(score), 1, _capi.stream_ptr()))
        p = torch.softmax(z[:, :V].double(), dim=-1)
        p[:, 1] = 0
        assert torch.equal(tok, (p / noise.double()).argmax(dim=-1))
