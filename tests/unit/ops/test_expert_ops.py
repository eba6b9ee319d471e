"""The ops of pre-norm decoders with routed experts, rotary attention, retention and matrix memories, each alone against the plain
functions of the Lefisun oracle: host versions in fp32, gfx950 kernels in fp32 and bf16."""
import math

import pytest
import torch

from deepspeedsyclsupport_amd.ops import expert_ops, hybrid_ops, mixer_ops

from ..inference.v2 import lefisun_oracle as O
from .test_hybrid_ops import CASES, GPU, _one_thread, _sub, close, meta, rnd  # noqa: F401


# ------------------------------------------------------------------------------------------------ residual
@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("W", [64, 132, 37, 520, 2048, 4096, 6000, 16384])
@pytest.mark.parametrize("T", [9, 600])
def test_pre_norm(device, dtype, tol, W, T):
    if T > 9 and (device == "cpu" or W == 6000):
        T = 10
    eps, mult, K = 1e-3, 0.02, 3
    w, fw = 1 + rnd(W, seed=4, scale=0.2), 1 + rnd(W, seed=7, scale=0.2)
    embed, ids = rnd(11, W, seed=5).to(dtype), (torch.arange(T) * 7 % 11).to(torch.int32)
    y = (rnd(T, W, seed=6) * 1e-2).to(dtype)       # of the order of eps: it counts
    d = [t.to(device) for t in (w, fw)]
    x = torch.full((T, W), float("nan"), device=device)
    norm = lambda s, g: O.rms(s, eps) * g.double()
    h = expert_ops.pre_norm(x, None, d[0], eps, ids=ids.to(device), embed=embed.to(device), mult=mult)
    want = embed.double()[ids.long()] * mult
    assert h.dtype == dtype
    close(x, want, 1e-7)
    close(h, norm(want, w), tol)
    h = expert_ops.pre_norm(x, y.to(device), d[0], eps)
    want = want + y.double()
    close(x, want, 1e-6)      # the residual stays fp32
    close(h, norm(want, w), tol)
    # a token's experts: in the token's order, and spread over rows
    e, g = (rnd(T * K, W, seed=8) * 0.1).to(dtype), torch.softmax(rnd(T, K, seed=9), -1)
    rows = torch.randperm(T * K, generator=torch.Generator().manual_seed(0)).view(T, K).to(torch.int32)
    picks = torch.tensor([8, 2, 2], dtype=torch.int32, device=device)
    for r in (None, rows):
        s = expert_ops.ExpertSum(e.to(device), g.to(device), None if r is None else r.to(device))
        add = (e.double()[torch.arange(T * K).view(T, K) if r is None else r.long()] * g.double()[..., None]).sum(1)
        close(s.sum(), add, tol)
        before = x.clone()
        h = expert_ops.pre_norm(x, s, d[1], eps, rows=picks)
        assert torch.equal(x, before)
        close(h, norm(want + add, fw)[[8, 2, 2]], tol)
        h = expert_ops.pre_norm(x, s, d[0], eps)
        want = want + add
        close(x, want, 2e-6)
        close(h, norm(want, w), tol)


# ------------------------------------------------------------------------------------------------ routed experts
ROUTES = [(12, 3, 3, 2, 64), (8, 2, 1, 1, 40), (16, 4, 4, 1, 320), (7, 7, 1, 1, 33), (64, 8, 8, 3, 256), (24, 1, 6, 2, 72),
          (160, 6, 8, 3, 96), (256, 10, 16, 5, 128), (9, 3, 9, 5, 24), (128, 4, 1, 1, 136)]


@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("E,top,groups,keep,W", ROUTES)
@pytest.mark.parametrize("T", [1, 21, 1100])
def test_route(device, dtype, tol, E, top, groups, keep, W, T):
    """Choices and weights, with experts that would be chosen but for their group, and the lists by expert."""
    if device == "cpu" and T > 21:
        pytest.skip("sizes of device kernels")
    h, r = rnd(T, W, seed=1).to(dtype), rnd(E, W, seed=2, scale=1.5 * W**-0.5).to(dtype)
    z = h.double() @ r.double().t()
    e, w = O.route(z, top, groups, keep)
    if E == 12 and T == 21:    # without the groups the choice would be another one
        assert any(set(a.tolist()) != set(b.tolist()) for a, b in zip(e, z.topk(top, -1).indices))
    if device == "cpu":
        from deepspeedsyclsupport_amd.ops import reference
        ge, gw = reference.route(h, r, top, groups, keep)
    else:
        from deepspeedsyclsupport_amd.ops.native import expert_ops as native
        ge, gw, offs, order, at = native().route(h.cuda(), r.cuda(), top, groups, keep, True)
        e2, w2, none = native().route(h.cuda(), r.cuda(), top, groups, keep, False)[:3]
        assert none is None and torch.equal(e2, ge) and torch.equal(w2, gw)
        flat, order, at, offs = ge.view(-1).cpu().long(), order.cpu().long(), at.view(-1).cpu().long(), offs.cpu()
        assert torch.equal(offs[1:], torch.bincount(flat, minlength=E).cumsum(0).int()) and offs[0] == 0
        assert torch.equal(order[at], torch.arange(T * top))
        for x in range(E):
            assert (flat[order[offs[x]:offs[x + 1]]] == x).all()
    full = torch.zeros(T, E).double().scatter_(1, e, w)
    got = torch.zeros(T, E).double().scatter_(1, ge.cpu().long(), gw.cpu().double())
    # (a close call may go either way: then the weights of both are nearly the same)
    same = (full > 0) == (got > 0)
    assert same.all(-1).float().mean() >= (1.0 if T < 100 else 0.99)
    assert (full - got)[same.all(-1)].abs().max() < 1e-5


SIZES = [(12, 3, 64, 96), (8, 2, 40, 24), (4, 1, 256, 200), (9, 4, 136, 72), (16, 6, 320, 128), (5, 2, 33, 27), (64, 8, 128, 64),
         (32, 3, 256, 128), (3, 2, 448, 192), (6, 5, 128, 320)]


@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("E,top,W,F", SIZES)
@pytest.mark.parametrize("T", [1, 2, 19, 130, 700])
@pytest.mark.parametrize("path", ["rows", "order", "library"])
def test_experts(device, dtype, tol, E, top, W, F, T, path, monkeypatch):
    """Weights row by row and in operand order: few rows (lists made in the products), lists streamed, tiles; the library's
    grouped product; experts without a token."""
    if device == "cpu" and (T > 19 or E > 16):
        pytest.skip("sizes of device kernels")
    if path != "rows" and (dtype != torch.bfloat16 or W % 64 or F % 64 or (path == "library" and (T < 130 or W % 128 or F % 128))):
        pytest.skip("no such path at these sizes")
    if path == "library":
        monkeypatch.setattr(expert_ops, "LIBRARY_ROWS", 0)
    g = 2 if E % 2 == 0 else 1
    h = rnd(T, W, seed=1).to(dtype)
    r = rnd(E, W, seed=2, scale=2 * W**-0.5).to(dtype)
    fc1, fc2 = rnd(E, 2 * F, W, seed=3, scale=W**-0.5).to(dtype), rnd(E, W, F, seed=4, scale=F**-0.5).to(dtype)
    dev = [t.to(device) for t in (h, r, fc1, fc2)]
    order = tuple(expert_ops.operand_order(t) for t in dev[2:]) if path == "order" else None
    got = expert_ops.experts(*dev, top, g, 1 if top <= E // g else g, order)
    e, w = O.route(h.double() @ r.double().t(), top, g, 1 if top <= E // g else g)
    x = h.double()
    want = torch.zeros(T, W).double()
    for i in range(E):
        mid = O.silu(x @ fc1[i, :F].double().t()) * (x @ fc1[i, F:].double().t())
        want += (w * (e == i)).sum(-1, keepdim=True) * (mid @ fc2[i].double().t())
    d = (got.sum().double().cpu() - want).abs().amax(-1) / want.abs().max()
    assert (d > 1.5 * tol).float().mean() <= (0 if T < 100 else 0.01), d.max()    # (close calls of the router)


@GPU
@pytest.mark.parametrize("path", ["rows", "stream", "tile"])
def test_experts_any_rows(path, monkeypatch):
    """Lists and products over row counts around every border of the paths; a single expert that takes everything."""
    E, top, W, F = 6, 2, 128, 192
    monkeypatch.setattr(expert_ops, "TILE_ROWS", 0 if path == "tile" else 1 << 20)
    r, fc1, fc2 = (rnd(*s, seed=i, scale=0.1).bfloat16().cuda() for i, s in enumerate([(E, W), (E, 2 * F, W), (E, W, F)]))
    for T in (15, 16, 17, 31, 33, 63, 65, 127, 128, 129, 255, 256, 257, 289, 511, 513):
        h = rnd(T, W, seed=T).bfloat16()
        h[:, 0] = 30.0
        r[:, 0] = torch.tensor([5.0, 0, 0, 2.0, 0, 0]).bfloat16()   # every token: experts 0 and 3
        order = None if path == "rows" else (expert_ops.operand_order(fc1), expert_ops.operand_order(fc2))
        got = expert_ops.experts(h.cuda(), r, fc1, fc2, top, order=order)
        x, want = h.double(), 0
        e, w = O.route(x @ r.double().cpu().t(), top, 1, 1)
        assert set(e.view(-1).tolist()) == {0, 3}
        for i in (0, 3):
            a = fc1[i].double().cpu()
            mid = O.silu(x @ a[:F].t()) * (x @ a[F:].t())
            want = want + (w * (e == i)).sum(-1, keepdim=True) * (mid @ fc2[i].double().cpu().t())
        close(got.sum(), want, 2e-2)


# ------------------------------------------------------------------------------------------------ rotary attention
@pytest.mark.parametrize("device", [pytest.param("cpu"), pytest.param("cuda", marks=GPU)])
def test_rope_table(device):
    """Angles of far positions, fp32 to the last digits."""
    pos = torch.tensor([0, 1, 17, 4095, 131071, 1000003], dtype=torch.int32)
    freq = torch.tensor([1e4**(-2 * i / 24) / 3 for i in range(12)], dtype=torch.float64)
    got = hybrid_ops.rope_table(pos.to(device), freq.to(device)).cpu()
    a = pos.double()[:, None] * freq
    close(got, torch.stack([a.cos(), a.sin()], -1), 3e-7)


@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("H,G,dk,dv,rot", [(6, 2, 32, 16, 16), (3, 3, 24, 40, 24), (4, 1, 64, 64, 0), (18, 2, 128, 128, 64),
                                           (2, 1, 20, 12, 6), (5, 5, 7, 9, 2), (12, 4, 96, 192, 48), (2, 2, 300, 8, 256)])
@pytest.mark.parametrize("chunk", [13, 0])
def test_rotary_attention(device, dtype, tol, H, G, dk, dv, rot, chunk):
    """Biases, norms over all heads, partial rotation, cache append and attention with a sink over scattered pages: two decodes,
    a fresh prompt and a continued portion in one batch; inputs and outputs are columns of wider rows."""
    eps, scale, mult, base = 1e-3, 1.5 * dk**-0.5, 0.6, 300.0
    lens = (30, 27, 40, 25)
    nq, nk, nv = H * dk, G * dk, G * dv
    N, pad = nq + nk + nv, 8
    bias, qw, kw = rnd(N, seed=3), 1 + rnd(nq, seed=1, scale=0.3), 1 + rnd(nk, seed=2, scale=0.3)
    sink = rnd(H, seed=4)
    sink[0] = 3.0
    qkv = [rnd(n, N + 2 * pad, seed=10 + i).to(dtype) for i, n in enumerate(lens)]
    freq = torch.tensor([base**(-2 * i / max(rot, 1)) for i in range(rot // 2)], dtype=torch.float64, device=device)
    m, nb = meta([(0, n) for n in lens], device)
    kc = torch.full((nb, G, 8, dk), 3.0, dtype=dtype, device=device)
    vc = torch.full((nb, G, 8, dv), 3.0, dtype=dtype, device=device)
    dev = [t.to(device) for t in (bias, qw, kw)]

    def run(rows, mm):
        x = torch.cat([qkv[i][a:b] for i, a, b in rows]).to(device)
        cs = hybrid_ops.rope_table(mm.pos_ids, freq) if rot else None
        q = hybrid_ops.qk_rope_append(x[:, pad:pad + N], *dev, eps, cs, mm, kc, vc, H, mult)
        out = torch.full((len(x), H * dv + 2 * pad), 9.0, dtype=dtype, device=device)
        hybrid_ops.ragged_attention(q, kc, vc, mm, scale, chunk=chunk, sink=sink.to(device), out=out[:, pad:pad + H * dv])
        assert (out[:, :pad] == 9).all() and (out[:, pad + H * dv:] == 9).all()
        return out[:, pad:pad + H * dv]

    portions = [(29, 1), (26, 1), (0, 40), (8, 17)]
    run([(0, 0, 29), (1, 0, 26), (3, 0, 8)], _sub(m, [0, 1, 3], [(0, 29), (0, 26), (0, 8)], device))
    got = run([(i, s, s + n) for i, (s, n) in enumerate(portions)], _sub(m, range(4), portions, device))
    want = []
    for i, (s, n) in enumerate(portions):
        x = qkv[i][:, pad:pad + N].double() + bias.double()
        q, k = O.rms(x[:, :nq], eps) * qw.double(), O.rms(x[:, nq:nq + nk], eps) * kw.double()
        turn = lambda y: O.rotate(y, rot, base)
        o = []
        for h in range(H):
            g = h // (H // G)
            o.append(_sunk(turn(q[:, h * dk:(h + 1) * dk]), turn(k[:, g * dk:(g + 1) * dk]),
                           mult * x[:, nq + nk + g * dv:nq + nk + (g + 1) * dv], scale, chunk, sink[h].double()))
        want.append(torch.stack(o, 1).reshape(-1, H * dv)[s:s + n])
    close(got, torch.cat(want), tol)


def _sunk(q, k, v, scale, chunk, sink):
    """The oracle's sink has a score of zero: any other one is a common shift of all scores."""
    extra = math.sqrt(1 / scale)
    q = torch.cat([q, torch.full((len(q), 1), extra)], 1).double()
    k = torch.cat([k, (torch.full((len(k), 1), extra) * -sink)], 1).double()
    return O.chunked_attention(q, k, v, scale, chunk)


@GPU
@pytest.mark.parametrize("dtype,tol", [(torch.float32, 2e-5), (torch.bfloat16, 2e-2)])
@pytest.mark.parametrize("chunk", [0, 700, 130])
def test_sink_over_long_context(dtype, tol, chunk):
    """Decoding split over many ranges of keys, and prompts over many tiles: the sink joins once."""
    H, G, d, n, scale = 4, 2, 64, 1500, 0.05
    q, k, v = rnd(n, H, d, seed=1).to(dtype), rnd(n, G, d, seed=2).to(dtype), rnd(n, G, d, seed=3).to(dtype)
    sink = torch.tensor([8.0, -30.0, 0.0, 40.0])
    for s0, new in ((n - 1, 1), (n - 1 - 70, 71)):
        m, nb = meta([(s0, new)], "cuda", block=64)
        kc, vc = (torch.zeros(nb, G, 64, d, dtype=dtype, device="cuda") for _ in range(2))
        for c, x in ((kc, k), (vc, v)):
            blk = m.block_tables[0].long().cpu()
            c.cpu()
            pages = torch.zeros(len(blk) * 64, G, d, dtype=dtype)
            pages[:n] = x
            c[blk.cuda()] = pages.view(len(blk), 64, G, d).transpose(1, 2).contiguous().cuda()
        got = hybrid_ops.ragged_attention(q[s0:].contiguous().cuda(), kc, vc, m, scale, chunk=chunk, sink=sink.cuda())
        for h in range(H):
            g = h // 2
            want = []
            for i in (s0, n - 1):
                lo = i // chunk * chunk if chunk else 0
                s = k[lo:i + 1, g].double() @ q[i, h].double() * scale
                mx = max(s.max().item(), sink[h].item())
                p = torch.exp(s - mx)
                want.append(p / (p.sum() + math.exp(sink[h] - mx)) @ v[lo:i + 1, g].double())
            close(got[[0, -1], h], torch.stack(want), tol * max(0.05, want[0].abs().max().item()))


# ------------------------------------------------------------------------------------------------ recurrences
HEADS = [(3, 16, 24), (2, 48, 64), (1, 64, 72), (4, 33, 20), (2, 128, 130), (2, 200, 40), (1, 256, 96), (1, 300, 8), (3, 7, 5)]


def _run_portions(f, proj, device, slot):
    """Three sequences in portions: prompts by chunks, short portions, decodes, in reused slots."""
    at, got = [0, 0, 0], [[], [], []]
    for step in ([(0, 100), (1, 3), (2, 17)], [(1, 1), (0, 2), (2, 16)], [(0, 1), (1, 66)], [(0, 47), (2, 7)]):
        mm, _ = meta([(at[i], n) for i, n in step], device, slots=[slot[i] for i, _ in step])
        o = f(torch.cat([proj[i][at[i]:at[i] + n] for i, n in step]).to(device), mm)
        row = 0
        for i, n in step:
            got[i].append(o[row:row + n])
            row, at[i] = row + n, at[i] + n
    assert at == [len(p) for p in proj]
    return [torch.cat(g) for g in got]


@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("H,dk,dv", HEADS)
def test_retention(device, dtype, tol, H, dk, dv):
    """Portions in reused slots; the state is held to fp64 far below 16-bit precision whatever the storage type: turned keys
    must not be rounded once more on their way into it."""
    rot, base, first, scale = dk // 2 // 2 * 2, 50.0, 16, dk**-0.5
    la = mixer_ops.ScanLayout(rows=first + H * (2 * dk + 2 * dv), q=first, k=first + H * dk, v=first + 2 * H * dk,
                              gate=first + H * (2 * dk + dv), Hk=H, H=H, dk=dk, dv=dv)
    proj = [rnd(n, la.rows, seed=i).to(dtype) for i, n in enumerate((150, 70, 40))]
    decay = torch.tensor([0.05, 1.0, 0.97, 0.9][:H], dtype=torch.float64)
    state = torch.full((3, H, dv, la.dks), 7.0, device=device)    # leftovers of an earlier owner
    state[..., dk:] = 0
    freq = torch.tensor([base**(-2 * i / max(rot, 1)) for i in range(rot // 2)], dtype=torch.float64, device=device)
    ld, slot = decay.log().float().to(device), (2, 0, 1)
    got = _run_portions(lambda x, mm: mixer_ops.retention(
        x, la, state, mm, ld, hybrid_ops.rope_table(mm.pos_ids, freq) if rot else None, scale), proj, device, slot)
    for i, x in enumerate(proj):
        x = x.double()
        part = lambda at, w: x[:, at:at + H * w].view(-1, H, w)
        q, k, v = part(la.q, dk), part(la.k, dk), part(la.v, dv)
        turn = lambda y: O.rotate(y, rot, base)
        o = [O.decayed_scan(turn(q[:, h]), turn(k[:, h]) * scale, v[:, h], decay[h]) for h in range(H)]
        close(got[i], torch.stack(o, 1).reshape(-1, H * dv), tol)
        for h in range(H):
            wt = decay[h]**torch.arange(len(x) - 1, -1, -1).double()
            close(state[slot[i], h, :, :dk], (v[:, h] * wt[:, None]).t() @ turn(k[:, h]), 2e-5)
    assert not state[..., dk:].any()


@GPU
@pytest.mark.parametrize("H,dk,dv,S,n", [(2, 64, 64, 3, 300), (16, 128, 128, 16, 130), (3, 96, 40, 2, 257), (12, 256, 64, 20, 100),
                                         (2, 256, 96, 1, 200), (1, 24, 16, 2, 129)])
def test_turned_read_out(H, dk, dv, S, n):
    """Read-outs of turned keys and queries by chunks (narrow and wide workgroups, both chunk lengths) equal those token by
    token to well below 16 bits before they are stored."""
    la = mixer_ops.ScanLayout(rows=H * (2 * dk + dv), q=0, k=H * dk, v=2 * H * dk, gate=0, Hk=H, H=H, dk=dk, dv=dv)
    proj = rnd(S * n, la.rows, seed=3).bfloat16().cuda()
    freq = torch.tensor([100.0**(-2 * i / dk) for i in range(dk // 2)], dtype=torch.float64, device="cuda")
    ld, outs = torch.full((H, ), -0.02, device="cuda"), []
    for step in (n, 16):
        state, out = torch.zeros(S, H, dv, dk, device="cuda"), torch.empty(S, n, H * dv, device="cuda")
        for at in range(0, n, step):
            c = min(step, n - at)
            mm, _ = meta([(at, c)] * S, "cuda", slots=range(S))
            x = proj.view(S, n, -1)[:, at:at + c].reshape(S * c, -1).contiguous()
            out[:, at:at + c] = mixer_ops.retention(x, la, state, mm, ld, hybrid_ops.rope_table(mm.pos_ids, freq),
                                                    1.0).view(S, c, -1).float()
        outs.append((out, state))
    (a, sa), (b, sb) = outs
    close(sa, sb.cpu(), 1e-5)
    assert (a - b).abs().max() <= 2**-8 * a.abs().max() and ((a - b) != 0).float().mean() < 0.05   # single roundings of the output


def _gates(la, proj, at, b, cap, H):
    x = proj.double()
    i = O.soft_cap(x[:, at:at + H] + b[0].double(), cap)
    return i, O.log_sigmoid(O.soft_cap(x[:, at + H:at + 2 * H] + b[1].double(), cap))


@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("H,dk,dv", HEADS)
def test_matrix_memory(device, dtype, tol, H, dk, dv):
    """Gates, running maximum, state and normaliser over portions in reused slots; gates far on both sides of the cap, a head
    that forgets everything and one that forgets nothing."""
    first, scale, cap = 8, dk**-0.5, 6.0
    gates = first + H * (2 * dk + 2 * dv)
    la = mixer_ops.ScanLayout(rows=gates + 2 * H + 3, q=first, k=first + H * dk, v=first + 2 * H * dk, gate=gates - H * dv, Hk=H,
                              H=H, dk=dk, dv=dv)
    proj = [rnd(n, la.rows, seed=i) for i, n in enumerate((150, 70, 40))]
    for p in proj:
        p[:, gates:gates + H] *= 3
        p[::7, gates] += 40                       # capped
        p[:, gates + H:gates + 2 * H] = p[:, gates + H:gates + 2 * H] * 2 + torch.tensor([0.0, 8.0, -7.0, 1.0])[:H]
    proj = [p.to(dtype) for p in proj]
    b = rnd(2, H, seed=9)
    slots = {"state": torch.full((3, H, dv, la.dks), 7.0, device=device), "peak": torch.full((3, H), 9.0, device=device),
             "norm": torch.full((3, H, -(-dv // 32), la.dks), -5.0, device=device)}
    for n in ("state", "norm"):
        slots[n][..., dk:] = 0
    d, slot = b.to(device), (2, 0, 1)
    got = _run_portions(lambda x, mm: mixer_ops.matrix_memory(x, la, slots, mm, gates, d[0], d[1], cap, scale), proj, device, slot)
    for i, x in enumerate(proj):
        li, lf = _gates(la, x, gates, b, cap, H)
        x = x.double()
        part = lambda at, w: x[:, at:at + H * w].view(-1, H, w)
        q, k, v = part(la.q, dk) * scale, part(la.k, dk), part(la.v, dv)
        want = torch.stack([O.matrix_memory(q[:, h], k[:, h], v[:, h], li[:, h], lf[:, h]) for h in range(H)], 1)
        # a denominator that nearly cancels magnifies rounding with its read-out: compare each token with its own size
        e = (got[i].double().cpu() - want.reshape(-1, H * dv)).view(-1, H, dv).abs().amax(-1)
        assert (e <= (tol if dtype != torch.float32 else 2e-4) * want.abs().amax(-1).clamp(min=1)).all()
        m = torch.zeros(H).double()
        for t in range(len(x)):
            m = torch.maximum(lf[t] + m, li[t])
        close(slots["peak"][slot[i]], m, 2e-5)
    assert not slots["state"][..., dk:].any() and not slots["norm"][..., dk:].any()
    assert (slots["norm"] == slots["norm"][:, :, :1]).all()     # every copy of the normaliser is the same


@GPU
@pytest.mark.parametrize("dk,dv", [(16, 16), (48, 64), (128, 80), (200, 64)])
def test_chunked_memory_is_fp32(dk, dv):
    """State and normaliser of the chunked form against fp64 at fp32 precision, and the same portions cut otherwise."""
    H, n, cap = 2, 333, 10.0
    gates = H * (2 * dk + 2 * dv)
    la = mixer_ops.ScanLayout(rows=gates + 2 * H, q=0, k=H * dk, v=2 * H * dk, gate=gates - H * dv, Hk=H, H=H, dk=dk, dv=dv)
    proj = rnd(n, la.rows, seed=3).bfloat16()
    proj[:, gates + H] += 6
    b = torch.zeros(2, H)
    li, lf = _gates(la, proj, gates, b, cap, H)
    x = proj.double()
    outs = []
    for cuts in ([n], [100, 64, 100, 69], [17] * 19 + [10], [1] * n):
        slots = {"state": torch.zeros(1, H, dv, la.dks, device="cuda"), "peak": torch.zeros(1, H, device="cuda"),
                 "norm": torch.zeros(1, H, -(-dv // 32), la.dks, device="cuda")}
        at, got = 0, []
        for c in cuts:
            mm, _ = meta([(at, c)], "cuda", slots=[0])
            got.append(mixer_ops.matrix_memory(proj[at:at + c].cuda(), la, slots, mm, gates, b[0].cuda(), b[1].cuda(), cap, dk**-0.5))
            at += c
        outs.append(torch.cat(got).float().cpu())
        for h in range(H):
            S, z, m = torch.zeros(dk, dv).double(), torch.zeros(dk).double(), torch.zeros(()).double()
            for t in range(n):
                k, v = x[t, la.k + h * dk:la.k + (h + 1) * dk], x[t, la.v + h * dv:la.v + (h + 1) * dv]
                new = torch.maximum(lf[t, h] + m, li[t, h])
                a, c = torch.exp(lf[t, h] + m - new), torch.exp(li[t, h] - new)
                S, z, m = a * S + c * k[:, None] * v, a * z + c * k, new
            close(slots["state"][0, h, :, :dk].t(), S, 3e-6)
            close(slots["norm"][0, h, 0, :dk], z, 3e-6)
    for o in outs[1:]:
        assert ((o - outs[0]).abs() <= 1.6e-2 * outs[0].abs() + 1e-3).all()


@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("P,parts", [(24, 3), (64, 5), (96, 4), (128, 16), (192, 2), (500, 1), (37, 2), (1024, 3), (8, 9)])
def test_gated_norm_of_heads(device, dtype, tol, P, parts):
    """Parts of a head's size, with and without a weight, into columns of a wider matrix."""
    T, eps, C, pad = 13, 1e-2, P * parts, 8
    y, proj, w = rnd(T, C, seed=1).to(dtype), rnd(T, C + 16, seed=2).to(dtype), 1 + rnd(C, seed=3, scale=0.3)
    y[:, P:] *= 5                       # unequal parts
    g = proj[:, 8:8 + C].double()
    normed = O.rms(y.double().view(T, parts, P), eps).view(T, C)
    for weight, mode, want in ((w, "sigmoid_after", normed * w.double() * O.sigmoid(g)), (None, "silu_after", normed * O.silu(g)),
                               (w, "silu_after", normed * w.double() * O.silu(g))):
        out = torch.full((T, C + 2 * pad), 9.0, dtype=dtype, device=device)
        mixer_ops.gated_norm(y.to(device), proj.to(device), 8, None if weight is None else weight.to(device), parts, eps, mode,
                             out[:, pad:pad + C])
        close(out[:, pad:pad + C], want, tol)
        assert (out[:, :pad] == 9).all() and (out[:, pad + C:] == 9).all()
