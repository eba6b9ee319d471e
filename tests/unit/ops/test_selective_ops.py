"""The ops of decoders with a gated sandwich residual, windowed attention, selective state spaces and plain routed experts, each
alone against the plain functions of the Nigilorn oracle: host versions in fp32, gfx950 kernels in fp32 and bf16."""
import pytest
import torch

from deepspeedsyclsupport_amd.inference.model_implementations.hybrid import Rotation
from deepspeedsyclsupport_amd.ops import expert_ops, hybrid_ops, mixer_ops

from ..inference.v2 import nigilorn_oracle as O
from .test_hybrid_ops import CASES, GPU, _one_thread, _sub, close, meta, rnd  # noqa: F401


# ------------------------------------------------------------------------------------------------ residual
@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("W", [64, 132, 37, 520, 2048, 4096, 6000, 16384])
@pytest.mark.parametrize("T", [9, 600])
def test_sandwich(device, dtype, tol, W, T):
    """Gate, norm of the output, sum, norm of the next input or none; outputs as they are and as experts beside a shared one."""
    if T > 9 and (device == "cpu" or W == 6000):
        T = 10
    eps, K, pad = 1e-3, 3, 8
    w, post, gate_b = 1 + rnd(W, seed=4, scale=0.2), 1 + rnd(W, seed=7, scale=0.2), rnd(W, seed=8)
    y, wide = (rnd(T, W, seed=6) * 1e-2).to(dtype), rnd(T, W + pad, seed=3).to(dtype)       # of the order of eps: it counts
    x0 = rnd(T, W, seed=5)
    x, d = x0.clone().to(device), [t.to(device) for t in (w, post, gate_b)]
    gate = wide.to(device)[:, pad:]
    g = O.sigmoid(wide[:, pad:].double() + gate_b.double())
    norm = lambda s, v: O.rms(s, eps) * v.double()
    h = expert_ops.pre_norm(x, y.to(device), d[0], eps, post_w=d[1], gate=gate, gate_b=d[2])
    want = x0.double() + norm(g * y.double(), post)
    assert h.dtype == dtype
    close(x, want, 2e-6)      # the residual stays fp32
    close(h, norm(want, w), tol)
    h = expert_ops.pre_norm(x, y.to(device), None, eps, post_w=d[1])      # no gate, no norm of the sum
    want = want + norm(y.double(), post)
    close(x, want, 2e-6)
    close(h, want, tol)
    e, wt, base = (rnd(T * K, W, seed=8) * 0.1).to(dtype), torch.softmax(rnd(T, K, seed=9), -1), (rnd(T, W, seed=10) * 0.1).to(dtype)
    rows = torch.randperm(T * K, generator=torch.Generator().manual_seed(0)).view(T, K).to(torch.int32)
    picks = torch.tensor([8, 2, 2], dtype=torch.int32, device=device)
    for r in (None, rows):
        s = expert_ops.ExpertSum(e.to(device), wt.to(device), None if r is None else r.to(device), base.to(device))
        add = (e.double()[torch.arange(T * K).view(T, K) if r is None else r.long()] * wt.double()[..., None]).sum(1) + base.double()
        close(s.sum(), add, tol)
        add = norm(g * add, post)
        before = x.clone()
        h = expert_ops.pre_norm(x, s, d[0], eps, rows=picks, post_w=d[1], gate=gate, gate_b=d[2])
        assert torch.equal(x, before)
        close(h, norm(want + add, w)[[8, 2, 2]], tol)
        h = expert_ops.pre_norm(x, s, d[0], eps, post_w=d[1], gate=gate, gate_b=d[2])
        want = want + add
        close(x, want, 4e-6)
        close(h, norm(want, w), tol)


@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("F,pad", [(64, 8), (45, 3), (24, 5)])
def test_row_act(device, dtype, tol, F, pad):
    x = rnd(7, 2 * F + pad, scale=2.0).to(dtype)
    d, g, u = x.to(device)[:, pad:], x[:, pad:pad + F].double(), x[:, pad + F:].double()
    close(expert_ops.row_act(d, "silu_glu"), O.silu(g) * u, tol)
    close(expert_ops.row_act(d[:, :F], "relu2"), torch.clamp(g, min=0)**2, tol)


# ------------------------------------------------------------------------------------------------ routed experts
@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("E,top,groups,keep,W", [(14, 4, 2, 1, 64), (12, 3, 3, 2, 40), (8, 2, 1, 1, 320), (7, 7, 1, 1, 33),
                                                 (64, 8, 8, 3, 256), (24, 1, 24, 6, 72), (160, 6, 8, 3, 96), (256, 10, 16, 5, 128)])
@pytest.mark.parametrize("T", [1, 21, 1100])
def test_route(device, dtype, tol, E, top, groups, keep, W, T):
    """Sigmoid scores, groups by their two best members (or their only one), weights times a factor."""
    if device == "cpu" and T > 21:
        pytest.skip("sizes of device kernels")
    h, r = rnd(T, W, seed=1).to(dtype), rnd(E, W, seed=2, scale=1.5 * W**-0.5).to(dtype)
    z = h.double() @ r.double().t()
    e, w = O.route(z, top, groups, keep, 1.9)
    if E in (12, 14) and T == 21:
        per = E // groups     # groups by their best member alone, or none at all, would choose otherwise
        s = O.sigmoid(z).view(T, groups, per)
        assert (s.amax(-1).topk(keep, -1).indices.sort(-1).values !=
                s.topk(2, -1).values.sum(-1).topk(keep, -1).indices.sort(-1).values).any()
        assert any(set(a.tolist()) != set(b.tolist()) for a, b in zip(e, z.topk(top, -1).indices))
    if device == "cpu":
        from deepspeedsyclsupport_amd.ops import reference
        ge, gw = reference.route(h, r, top, groups, keep, 1, 2, 1.9)
    else:
        from deepspeedsyclsupport_amd.ops.native import expert_ops as native
        ge, gw, offs, order, at = native().route(h.cuda(), r.cuda(), top, groups, keep, True, 1, 2, 1.9)
        flat, offs = ge.view(-1).cpu().long(), offs.cpu()
        assert torch.equal(offs[1:], torch.bincount(flat, minlength=E).cumsum(0).int())
        assert torch.equal(order.cpu().long()[at.view(-1).cpu().long()], torch.arange(T * top))
    full = torch.zeros(T, E).double().scatter_(1, e, w)
    got = torch.zeros(T, E).double().scatter_(1, ge.cpu().long(), gw.cpu().double())
    same = ((full > 0) == (got > 0)).all(-1)       # (a close call may go either way)
    assert same.float().mean() >= (1.0 if T < 100 else 0.99)
    assert (full - got)[same].abs().max() < 2e-5


@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("E,top,W,F", [(10, 3, 64, 112), (8, 2, 40, 24), (4, 1, 256, 200), (16, 6, 320, 128), (5, 2, 33, 27),
                                       (64, 8, 128, 64), (32, 3, 256, 128), (6, 5, 128, 320)])
@pytest.mark.parametrize("T", [1, 2, 19, 130, 700])
@pytest.mark.parametrize("path", ["rows", "order", "library"])
def test_plain_experts(device, dtype, tol, E, top, W, F, T, path, monkeypatch):
    """Two maps with a squared relu between, over every path of the products; a base beside the sum."""
    if device == "cpu" and (T > 19 or E > 16):
        pytest.skip("sizes of device kernels")
    if path != "rows" and (dtype != torch.bfloat16 or W % 64 or F % 64 or (path == "library" and (T < 130 or W % 128 or F % 128))):
        pytest.skip("no such path at these sizes")
    if path == "library":
        monkeypatch.setattr(expert_ops, "LIBRARY_ROWS", 0)
    g = 2 if E % 2 == 0 else 1
    keep = 1 if top <= E // g else g
    h, r = rnd(T, W, seed=1).to(dtype), rnd(E, W, seed=2, scale=2 * W**-0.5).to(dtype)
    fc1, fc2 = rnd(E, F, W, seed=3, scale=W**-0.5).to(dtype), rnd(E, W, F, seed=4, scale=F**-0.5).to(dtype)
    base = rnd(T, W, seed=5).to(dtype)
    dev = [t.to(device) for t in (h, r, fc1, fc2)]
    order = tuple(expert_ops.operand_order(t) for t in dev[2:]) if path == "order" else None
    got = expert_ops.experts(*dev, top, g, keep, order, score="sigmoid", best=2, scale=1.3, act="relu2")
    got.base = base.to(device)
    x = h.double()
    e, w = O.route(x @ r.double().t(), top, g, keep, 1.3)
    want = base.double()
    for i in range(E):
        mid = torch.clamp(x @ fc1[i].double().t(), min=0)**2
        want = want + (w * (e == i)).sum(-1, keepdim=True) * (mid @ fc2[i].double().t())
    d = (got.sum().double().cpu() - want).abs().amax(-1) / want.abs().max()
    assert (d > 1.5 * tol).float().mean() <= (0 if T < 100 else 0.01), d.max()    # (close calls of the router)


# ------------------------------------------------------------------------------------------------ rotation
@pytest.mark.parametrize("dims,base,factor,original,fast,slow", [
    (64, 500000.0, 4.0, 4096, 32.0, 1.0), (16, 30000.0, 2.0, 512, 24.0, 1.0), (8, 100.0, 8.0, 40, 4.0, 0.5), (2, 1e4, 3.0, 100, 8.0, 1.0),
    (32, 1e6, 1.0, 64, 64.0, 2.0), (6, 50.0, 16.0, 4000, 2.0, 1.5)])
def test_yarn_frequencies(dims, base, factor, original, fast, slow):
    """Frequencies and the factor of cosine and sine, with ramps inside, at either end and empty; angles from the shared table."""
    rot = O.rotation(dims, base, factor, original, fast, slow)
    f, grow = O.yarn(rot)
    r = Rotation({**rot, "scaling": {**rot["scaling"], "type": "yarn"}}, dims)
    got = r.frequencies("cpu")
    assert (got - torch.tensor(f, dtype=torch.float64)).abs().max() < 1e-14 and abs(r.mult - grow) < 1e-14
    pos = torch.tensor([0, 1, 17, 4095, 131071], dtype=torch.int32)
    a = pos.double()[:, None] * torch.tensor(f, dtype=torch.float64)
    for device in ["cpu"] + (["cuda"] if torch.cuda.is_available() else []):
        close(hybrid_ops.rope_table(pos.to(device), got.to(device), r.mult), grow * torch.stack([a.cos(), a.sin()], -1), 4e-7)


# ------------------------------------------------------------------------------------------------ windowed attention
@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("H,G,dk,dv,rot", [(6, 2, 32, 16, 16), (3, 3, 24, 40, 24), (4, 1, 64, 64, 0), (18, 2, 128, 128, 64),
                                           (2, 1, 20, 12, 6), (5, 5, 7, 9, 2), (12, 4, 96, 192, 44), (2, 2, 300, 8, 256),
                                           (8, 4, 120, 56, 10)])
@pytest.mark.parametrize("window", [13, 1, 0])
def test_window_attention(device, dtype, tol, H, G, dk, dv, rot, window):
    """Rotation of neighbours, then norms head by head, cache append and attention with a gate per head over scattered pages: two
    decodes, a fresh prompt and a continued portion in one batch; inputs are columns of wider rows."""
    eps, scale = 1e-2, 1.5 * dk**-0.5
    lens = (30, 27, 40, 25)
    nq, nk, nv = H * dk, G * dk, G * dv
    N, pad = nq + nk + nv, 8
    qkv = [rnd(n, N + H + pad, seed=10 + i).to(dtype) for i, n in enumerate(lens)]
    for x in qkv:
        x[:, pad:pad + nq + nk] *= 0.3     # the norm's eps counts
    r = O.rotation(rot or 2, 300.0, 5.0, 30)
    rotation = Rotation({**r, "dims": rot, "scaling": {**r["scaling"], "type": "yarn"}}, dk)
    freq = rotation.frequencies(device)
    m, nb = meta([(0, n) for n in lens], device)
    kc = torch.full((nb, G, 8, dk), 3.0, dtype=dtype, device=device)
    vc = torch.full((nb, G, 8, dv), 3.0, dtype=dtype, device=device)

    def run(rows, mm):
        x = torch.cat([qkv[i][a:b] for i, a, b in rows]).to(device)
        cs = hybrid_ops.rope_table(mm.pos_ids, freq, rotation.mult) if rot else None
        q = hybrid_ops.qk_norm_append(x[:, pad:pad + N], None, None, eps, None, None, mm.pos_ids, mm.seq_ids, mm.block_tables, kc,
                                      vc, H, cs)
        return hybrid_ops.ragged_attention(q, kc, vc, mm, scale, window=window, gate=x[:, pad + N:])

    portions = [(29, 1), (26, 1), (0, 40), (8, 17)]
    run([(0, 0, 29), (1, 0, 26), (3, 0, 8)], _sub(m, [0, 1, 3], [(0, 29), (0, 26), (0, 8)], device))
    got = run([(i, s, s + n) for i, (s, n) in enumerate(portions)], _sub(m, range(4), portions, device))
    want = []
    for i, (s, n) in enumerate(portions):
        x = qkv[i][:, pad:].double()
        turn = lambda y: O.rms(O.rotate(y, r) if rot else y, eps)
        o = []
        for h in range(H):
            g = h // (H // G)
            o.append(O.window_attention(turn(x[:, h * dk:(h + 1) * dk]), turn(x[:, nq + g * dk:nq + (g + 1) * dk]),
                                        x[:, nq + nk + g * dv:nq + nk + (g + 1) * dv], scale, window or 1000))
        want.append((torch.stack(o, 1) * O.sigmoid(x[:, N:])[..., None])[s:s + n])
    close(got, torch.cat(want), tol)


@GPU
@pytest.mark.parametrize("dtype,tol", [(torch.float32, 2e-5), (torch.bfloat16, 2e-2)])
@pytest.mark.parametrize("window", [0, 700, 130, 64])
def test_gate_over_long_context(dtype, tol, window):
    """Decoding split over many ranges of keys, and prompts over many tiles: the gate is applied once."""
    H, G, d, n, scale = 4, 2, 64, 1500, 0.05
    q, k, v = rnd(n, H, d, seed=1).to(dtype), rnd(n, G, d, seed=2).to(dtype), rnd(n, G, d, seed=3).to(dtype)
    gate = rnd(n, H, seed=4, scale=3.0).to(dtype)
    for s0, new in ((n - 1, 1), (n - 1 - 70, 71)):
        m, nb = meta([(s0, new)], "cuda", block=64)
        kc, vc = (torch.zeros(nb, G, 64, d, dtype=dtype, device="cuda") for _ in range(2))
        for c, x in ((kc, k), (vc, v)):
            blk = m.block_tables[0].long()
            pages = torch.zeros(len(blk) * 64, G, d, dtype=dtype)
            pages[:n] = x
            c[blk] = pages.view(len(blk), 64, G, d).transpose(1, 2).contiguous().cuda()
        got = hybrid_ops.ragged_attention(q[s0:].contiguous().cuda(), kc, vc, m, scale, window=window, gate=gate[s0:].cuda())
        for h in range(H):
            want = []
            for i in (s0, n - 1):
                lo = max(i - window + 1, 0) if window else 0
                p = torch.softmax(k[lo:i + 1, h // 2].double() @ q[i, h].double() * scale, -1)
                want.append(p @ v[lo:i + 1, h // 2].double() * O.sigmoid(gate[i, h].double()))
            close(got[[0, -1], h], torch.stack(want), tol * max(0.05, want[0].abs().max().item()))


# ------------------------------------------------------------------------------------------------ windowed latent attention
LATENTS = [(3, 16, 8, 24, 40), (2, 32, 16, 32, 64), (5, 20, 6, 12, 18), (16, 128, 64, 128, 512), (1, 8, 8, 8, 8), (4, 72, 24, 88, 48),
           (6, 24, 24, 40, 256)]


@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("dims", LATENTS)
@pytest.mark.parametrize("window", [0, 9, 70])
def test_window_latent_attention(device, dtype, tol, dims, window):
    """Queries straight from a wide projection row, no sink, a window and a factor of cosine and sine: two decodes, short and long
    continued portions and fresh prompts in one batch, contexts of which the window leaves only the end."""
    H, d, r, e, R = dims
    if device == "cpu" and R > 256:
        pytest.skip("sizes of device kernels")
    scale, eps, lens, Q = 1.5 * (d + r)**-0.5, 1e-3, (30, 190, 40, 90, 100, 330), H * (d + r)
    rot = O.rotation(r, 500.0, 3.0, 30)
    kn = 1 + rnd(R, seed=1, scale=0.2)
    uk, uv = rnd(H * d, R, seed=2, scale=R**-0.5).to(dtype), rnd(H * e, R, seed=3, scale=R**-0.5).to(dtype)
    rows = [rnd(n, Q + R + r + 8, seed=20 + i).to(dtype) for i, n in enumerate(lens)]
    want = []
    for x in rows:
        x = x.double()
        c = O.rms(x[:, Q:Q + R], eps) * kn.double()
        kr = O.rotate(x[:, Q + R:Q + R + r], rot)
        k, v = (c @ uk.double().t()).view(-1, H, d), (c @ uv.double().t()).view(-1, H, e)
        q = x[:, :Q].view(-1, H, d + r)
        want.append(torch.stack([O.window_attention(torch.cat([q[:, h, :d], O.rotate(q[:, h, d:], rot)], -1),
                                                    torch.cat([k[:, h], kr], -1), v[:, h], scale, window or 10000)
                                 for h in range(H)], 1))
    # the kernels turn halves: rows of pairs of neighbours are laid out so
    turned = torch.cat([torch.arange(0, r, 2), torch.arange(1, r, 2)])
    inner = torch.cat([torch.arange(d), d + turned])
    heads = (torch.arange(H)[:, None] * (d + r) + inner).flatten()
    at = torch.cat([heads, torch.arange(Q, Q + R), Q + R + turned, torch.arange(Q + R + r, Q + R + r + 8)])
    rows = [x[:, at].contiguous() for x in rows]
    rotation = Rotation({**rot, "scaling": {**rot["scaling"], "type": "yarn"}}, r)
    freq = rotation.frequencies(device)
    m, nb = meta([(0, n) for n in lens], device)
    lat = torch.full((nb, 1, 8, R + r), 3.0, dtype=dtype, device=device)
    ukv, ukt = torch.cat([uk, uv]).to(device), uk.view(H, d, R).transpose(1, 2).contiguous().to(device)

    def run(parts, mm):
        x = torch.cat([rows[i][a:b] for i, a, b in parts]).to(device)
        assert mixer_ops.latent_prepare(x[:, Q:Q + R + r], None, kn.to(device), eps, freq, mm, lat, 0, rotation.mult) is None
        return mixer_ops.latent_attention(x[:, :Q].unflatten(1, (H, d + r)), lat, ukv, ukt, freq, None, mm, scale, d, e, window,
                                          rotation.mult)

    portions = [(29, 1), (189, 1), (0, 40), (73, 17), (0, 100), (230, 100)]
    before = [(i, s) for i, (s, _) in enumerate(portions) if s]
    run([(i, 0, s) for i, s in before], _sub(m, [i for i, _ in before], [(0, s) for _, s in before], device))
    got = run([(i, s, s + n) for i, (s, n) in enumerate(portions)], _sub(m, range(6), portions, device))
    close(got, torch.cat([want[i][s:s + n] for i, (s, n) in enumerate(portions)]), tol)


# ------------------------------------------------------------------------------------------------ selective recurrences
SCANS = [(48, 12, 4), (64, 16, 4), (40, 5, 1), (33, 7, 3), (336, 20, 2), (130, 64, 5), (512, 16, 4), (100, 33, 6), (16, 200, 4),
         (66, 128, 4), (24, 1, 2), (8, 256, 3)]


@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("C,N,taps", SCANS)
def test_selective_scan(device, dtype, tol, C, N, taps):
    """Convolution and recurrence over portions in reused slots: prompts, short portions, decodes; steps from tiny to several units;
    numbers that hardly decay beside some that vanish at once. The state is held to fp32."""
    if device == "cpu" and C * N > 9000:
        pytest.skip("sizes of device kernels")
    pad, lens = 8, (150, 70, 45)
    proj = [rnd(n, 2 * C + pad, seed=i).to(dtype) for i, n in enumerate(lens)]
    w, b, skip = rnd(C, taps, seed=5, scale=0.5), rnd(C, seed=6, scale=0.3), rnd(C, seed=7)
    dt = [(rnd(n, C, seed=10 + i) * 2).to(dtype) for i, n in enumerate(lens)]
    low = [rnd(n, 2 * N + pad, seed=20 + i).to(dtype) for i, n in enumerate(lens)]
    dt_b, a_log = rnd(C, seed=8) - 3, rnd(C, N, seed=9) * 2 - 1
    a_log[0], a_log[-1] = -9.0, 4.0
    decay = -torch.exp(a_log)
    state = torch.full((3, C, -(-N // 4) * 4), 7.0, device=device)    # leftovers of an earlier owner
    conv = torch.full((3, taps - 1, C), 5.0, dtype=dtype, device=device) if taps > 1 else None
    dev = [t.to(device) for t in (w, b, dt_b, decay, skip)]
    slot, at, got = (2, 0, 1), [0, 0, 0], [[], [], []]
    for step in ([(0, 100), (1, 3), (2, 17)], [(1, 1), (0, 2), (2, 16)], [(0, 1), (1, 66)], [(0, 47), (2, 11)], [(2, 1)]):
        mm, _ = meta([(at[i], n) for i, n in step], device, slots=[slot[i] for i, _ in step])
        part = lambda x: torch.cat([x[i][at[i]:at[i] + n] for i, n in step]).to(device)
        p, l = part(proj), part(low)
        x = mixer_ops.causal_conv(p[:, pad:pad + C], dev[0], dev[1], conv, mm)
        y = mixer_ops.selective_scan(x, part(dt), l[:, pad:], p[:, pad + C:], *dev[2:], state, p[:, pad:pad + C], conv, mm)
        row = 0
        for i, n in step:
            got[i].append((x[row:row + n], y[row:row + n]))
            row, at[i] = row + n, at[i] + n
    assert at == list(lens)
    for i in range(3):
        p = proj[i].double()
        x = O.silu(O.causal_conv(p[:, pad:pad + C], w.double(), b.double()))
        close(torch.cat([a for a, _ in got[i]]), x, tol)
        if dtype == torch.bfloat16:
            x = torch.cat([a for a, _ in got[i]]).double().cpu()     # (as it was stored)
        s = O.softplus(dt[i].double() + dt_b.double())
        B, Cn = low[i][:, pad:].double().split(N, -1)
        y = (O.selective_scan(x, s, decay.double(), B, Cn) + skip.double() * x) * O.silu(p[:, pad + C:])
        close(torch.cat([a for _, a in got[i]]), y, tol)
        keep = torch.exp(decay.double()[None] * (s.sum(0) - s.cumsum(0))[..., None])     # [n, C, N]: what the last state keeps
        want = (keep * (s * x)[..., None] * B[:, None]).sum(0)
        close(state[slot[i], :, :N], want, 3e-5)
        if taps > 1:
            assert torch.equal(conv[slot[i]].cpu(), proj[i][-(taps - 1):, pad:pad + C])


@GPU
@pytest.mark.parametrize("dtype,tol", [(torch.float32, 2e-5), (torch.bfloat16, 2e-2)])
@pytest.mark.parametrize("C,N,S", [(2048, 16, 12), (4096, 16, 1), (1024, 24, 24), (1024, 64, 8), (256, 128, 2)])
def test_selective_scan_wide(dtype, tol, C, N, S):
    """Sizes that choose every number of lanes per channel: equal to the same tokens one by one."""
    n, T = 75, 75 * S
    x, z, dt, low = (rnd(T, c, seed=i).to(dtype).cuda() for i, c in enumerate((C, C, C, 2 * N)))
    dt_b, decay, skip = rnd(C, seed=8).cuda() - 3, -torch.exp(rnd(C, N, seed=9)).cuda(), rnd(C, seed=7).cuda()
    outs = []
    for step in (n, 1):
        state, out = torch.full((S, C, N), 3.0, device="cuda"), torch.empty(S, n, C, device="cuda")
        for at in range(0, n, step):
            c = min(step, n - at)
            mm, _ = meta([(at, c)] * S, "cuda", slots=range(S))
            part = lambda v: v.view(S, n, -1)[:, at:at + c].reshape(S * c, -1).contiguous()
            xp = part(x)
            out[:, at:at + c] = mixer_ops.selective_scan(xp, part(dt), part(low), part(z), dt_b, decay, skip, state, xp, None,
                                                         mm).view(S, c, C).float()
        outs.append((out, state))
    (a, sa), (b, sb) = outs
    close(sa, sb.cpu(), 1e-5)
    assert (a - b).abs().max() <= (2**-8 if dtype == torch.bfloat16 else 1e-5) * a.abs().max()
