"""Each op of `ops/mixer_ops.py` alone, against the plain functions of the Perelorn oracle: host versions in fp32, gfx950
kernels in fp32 and bf16."""
import pytest
import torch

from deepspeedsyclsupport_amd.ops import hybrid_ops, mixer_ops as ops

from ..inference.v2 import perelorn_oracle as O
from .test_hybrid_ops import CASES, GPU, _one_thread, _sub, close, meta, rnd  # noqa: F401


@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("W", [64, 132, 37, 520, 2048, 4096, 6000, 16384])
@pytest.mark.parametrize("T", [9, 600])
def test_post_norm(device, dtype, tol, W, T):
    if T > 9 and (device == "cpu" or W == 6000):
        T = 10
    eps, mult = 1e-3, 1.7
    w, fw = 1 + rnd(W, seed=4, scale=0.2), 1 + rnd(W, seed=7, scale=0.2)
    embed, ids = rnd(11, W, seed=5).to(dtype), (torch.arange(T) * 7 % 11).to(torch.int32)
    y = (rnd(T, W, seed=6) * 1e-2).to(dtype)       # of the order of eps: it counts
    d = [t.to(device) for t in (w, fw)]
    x = torch.full((T, W), float("nan"), device=device)
    h = ops.post_norm(x, None, None, 0.0, ids=ids.to(device), embed=embed.to(device))
    assert h.dtype == dtype and torch.equal(h.cpu(), embed[ids.long()])
    close(x, embed[ids.long()], 0.0)
    h = ops.post_norm(x, y.to(device), d[0], eps)
    want = embed.double()[ids.long()] + O.rms_norm(y.double(), w.double(), eps)
    close(x, want, 1e-6)      # the residual stays fp32
    close(h, want, tol)
    rows = torch.tensor([8, 2, 2], dtype=torch.int32, device=device)
    before = x.clone()
    h = ops.post_norm(x, y.to(device), d[0], eps, rows=rows, final_w=d[1], mult=mult)
    assert torch.equal(x, before)
    want = O.rms_norm(want + O.rms_norm(y.double(), w.double(), eps), fw.double(), eps) * mult
    close(h, want[[8, 2, 2]], tol)


@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("C,parts,shift", [(96, 4, 8), (96, 1, 8), (90, 6, 3), (37, 1, 0), (4096, 1, 16), (2048, 2, 64),
                                           (7168, 1, 8), (12288, 1, 8), (20000, 1, 8)])
def test_gated_norm(device, dtype, tol, C, parts, shift):
    T, eps = 7, 1e-2
    y, proj, w = rnd(T, C, seed=1).to(dtype), rnd(T, C + 2 * shift, seed=2).to(dtype), 1 + rnd(C, seed=3, scale=0.3)
    y[:, C // parts:] *= 5                       # unequal parts
    g = proj[:, shift:shift + C].double()
    args = (y.to(device), proj.to(device), shift, w.to(device), parts, eps)
    close(ops.gated_norm(*args, "silu_before"), O.grouped_rms(y.double() * O.silu(g), parts, eps) * w.double(), tol)
    close(ops.gated_norm(*args, "sigmoid_after"), O.grouped_rms(y.double(), parts, eps) * w.double() * O.sigmoid(g), tol)


@pytest.mark.parametrize("device,dtype,tol", CASES)
def test_gelu_and_token_gate(device, dtype, tol):
    x = rnd(5, 77, scale=2.0).to(dtype)
    close(ops.gelu(x.to(device)), O.gelu_erf(x.double()), tol)
    table, ids = rnd(6, 3 * 77, seed=1).to(dtype), torch.tensor([5, 0, 3, 3, 1], dtype=torch.int32)
    for first in (0, 77, 154):
        want = O.gelu_tanh(x.double()) * table.double()[ids.long(), first:first + 77]
        close(ops.token_gate(x.to(device), ids.to(device), table.to(device), first), want, tol)


@GPU
@pytest.mark.parametrize("rows", [1, 2, 5, 16, 40])
@pytest.mark.parametrize("N,K", [(96, 64), (513, 320), (90, 256), (33, 24), (1024, 2048)])
def test_product_with_gelu(rows, N, K):
    """The activation as an epilogue of the decode streams."""
    from deepspeedsyclsupport_amd.ops.bf16_gemv import Bf16Weight
    x, w = rnd(rows, K).bfloat16().cuda(), rnd(N, K, seed=1, scale=K**-0.5).bfloat16().cuda()
    plain = x.double().cpu() @ w.double().cpu().t()
    sh = Bf16Weight(w) if Bf16Weight.supported(w) else None
    for s in (None, sh):
        close(hybrid_ops.linear(x, w, s, act="gelu"), O.gelu_erf(plain), 1e-2)
        close(hybrid_ops.linear(x, w, s), plain, 1e-2)     # the epilogue leaves the sums cleared


# ------------------------------------------------------------------------------------------------ latent attention
DIMS = [(3, 16, 8, 24, 40, 32), (8, 32, 16, 32, 96, 48), (2, 12, 6, 10, 20, 18), (16, 64, 32, 64, 256, 64),
        (5, 128, 64, 128, 512, 40), (40, 40, 8, 72, 136, 24), (1, 8, 2, 8, 8, 8)]


def latent_layer_inputs(dims, lens, dtype, seed=0):
    H, d, r, e, R, Q = dims
    w = {n: t.to(dtype) for n, t in {
        "uk": rnd(H * d, R, seed=seed + 1, scale=R**-0.5), "uv": rnd(H * e, R, seed=seed + 2, scale=R**-0.5)}.items()}
    w["qn"], w["kn"], w["sink"] = 1 + rnd(Q, seed=3, scale=0.2), 1 + rnd(R, seed=4, scale=0.2), rnd(H, seed=5)
    down = [rnd(n, Q + R + r, seed=10 + i).to(dtype) for i, n in enumerate(lens)]
    q = [(1.5 * rnd(n, H, d + r, seed=20 + i)).to(dtype) for i, n in enumerate(lens)]
    return w, down, q


def latent_want(dims, w, down, q, base, scale, eps):
    H, d, r, e, R, Q = dims
    x = down.double()
    c = O.rms_norm(x[:, Q:Q + R], w["kn"].double(), eps)
    kr = O.rotate(x[:, Q + R:], r, base)
    k, v = (c @ w["uk"].double().t()).view(-1, H, d), (c @ w["uv"].double().t()).view(-1, H, e)
    out = []
    for h in range(H):
        qh = torch.cat([q[:, h, :d].double(), O.rotate(q[:, h, d:].double(), r, base)], -1)
        out.append(O.sink_attention(qh, torch.cat([k[:, h], kr], -1), v[:, h], scale, w["sink"][h].double()))
    return O.rms_norm(x[:, :Q], w["qn"].double(), eps), torch.stack(out, 1)


@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("dims", DIMS)
def test_latent_attention(device, dtype, tol, dims):
    """Norms, rotation, cache append and attention over scattered pages: two decodes, a short and a long continued portion
    and two fresh prompts (one short) in one batch."""
    H, d, r, e, R, Q = dims
    if device == "cpu" and R > 256:
        pytest.skip("sizes of device kernels")
    base, scale, eps = 500.0, (d + r)**-0.5, 1e-3
    lens = (30, 17, 40, 25, 100, 130)
    w, down, q = latent_layer_inputs(dims, lens, dtype)
    want = [latent_want(dims, w, x, y, base, scale, eps) for x, y in zip(down, q)]
    m, nb = meta([(0, n) for n in lens], device)
    lat = torch.full((nb, 1, 8, R + r), 3.0, dtype=dtype, device=device)
    dev = {n: t.to(device) for n, t in w.items()}
    ukv = torch.cat([dev["uk"], dev["uv"]])
    ukt = dev["uk"].view(H, d, R).transpose(1, 2).contiguous()
    freq = torch.tensor([base**(-2 * i / r) for i in range(r // 2)], dtype=torch.float64, device=device)

    def run(rows, mm):
        x = torch.cat([down[i][a:b] for i, a, b in rows]).to(device)
        cq = ops.latent_prepare(x, dev["qn"], dev["kn"], eps, freq, mm, lat, Q)
        close(cq, torch.cat([want[i][0][a:b] for i, a, b in rows]), tol)
        return ops.latent_attention(torch.cat([q[i][a:b] for i, a, b in rows]).to(device), lat, ukv, ukt, freq, dev["sink"], mm,
                                    scale, d, e)

    # everything but the last portions first, then the batch under test (kernel order: decodes, short, long)
    portions = [(29, 1), (16, 1), (0, 40), (8, 17), (0, 100), (33, 97)]
    run([(0, 0, 29), (1, 0, 16), (3, 0, 8), (5, 0, 33)], _sub(m, [0, 1, 3, 5], [(0, 29), (0, 16), (0, 8), (0, 33)], device))
    got = run([(i, s, s + n) for i, (s, n) in enumerate(portions)], _sub(m, range(6), portions, device))
    close(got, torch.cat([want[i][1][s:s + n] for i, (s, n) in enumerate(portions)]), tol)


@GPU
@pytest.mark.parametrize("dtype,tol", [(torch.float32, 2e-5), (torch.bfloat16, 2e-2)])
@pytest.mark.parametrize("H,n_new", [(2, 1), (24, 1), (6, 3), (20, 9), (2, 70)])
def test_latent_long_context(dtype, tol, H, n_new):
    """A far key that dominates its query, contexts over many ranges and pages, sinks that take most of the weight."""
    dims = (H, 32, 16, 32, 64, 16)
    _, d, r, e, R, Q = dims
    base, scale, eps, device, n = 1e4, 0.3, 1e-5, "cuda", 900
    w, down, q = latent_layer_inputs(dims, (n, ), dtype, seed=40)
    w["sink"][0] += 6
    # the last queries look at key 5: the query of head h is that head's key of token 5
    x = down[0].double()
    c5 = O.rms_norm(x[5:6, Q:Q + R], w["kn"].double(), eps)
    q[0][-1, :, :d] = (4 * (c5 @ w["uk"].double().t()).view(H, d)).to(dtype)
    _, want = latent_want(dims, w, down[0], q[0], base, scale, eps)
    m, nb = meta([(0, n)], device)
    lat = torch.zeros(nb, 1, 8, R + r, dtype=dtype, device=device)
    dev = {k: t.to(device) for k, t in w.items()}
    ukv, ukt = torch.cat([dev["uk"], dev["uv"]]), dev["uk"].view(H, d, R).transpose(1, 2).contiguous()
    freq = torch.tensor([base**(-2 * i / r) for i in range(r // 2)], dtype=torch.float64, device=device)
    got = []
    for s, k in ((0, n - n_new), (n - n_new, n_new)):
        mm = _sub(m, [0], [(s, k)], device)
        ops.latent_prepare(down[0][s:s + k].to(device), dev["qn"], dev["kn"], eps, freq, mm, lat, Q)
        got.append(ops.latent_attention(q[0][s:s + k].to(device), lat, ukv, ukt, freq, dev["sink"], mm, scale, d, e))
    close(got[1], want[-n_new:], tol)
    close(got[0], want[:-n_new], tol)
    assert (want[-1] - want[-2]).abs().max() > 20 * tol


@pytest.mark.parametrize("device,dtype,tol", CASES)
def test_rotation_far_out(device, dtype, tol):
    """Angles keep their digits at positions of a hundred thousand."""
    r, p0, base = 8, 131000, 50.0
    freq = torch.tensor([base**(-2 * i / r) for i in range(r // 2)], dtype=torch.float64, device=device)
    R, Q = 8, 8
    down = rnd(3, Q + R + r, seed=1).to(dtype)
    m, _ = meta([(0, 3)], device)
    lat = torch.zeros(8, 1, 8, R + r, dtype=dtype, device=device)
    m.pos_ids = torch.tensor([p0, p0 + 1, p0 + 2], dtype=torch.int32, device=device)
    m.block_tables = (torch.arange(p0 // 8 + 2, dtype=torch.int32, device=device) % 8)[None].contiguous()
    ops.latent_prepare(down.to(device), torch.ones(Q, device=device), torch.ones(R, device=device), 1e-6, freq, m, lat, Q)
    want = O.rotate(down[:, Q + R:].double(), r, base, first=p0)
    got = torch.stack([lat[(p // 8) % 8, 0, p % 8, R:] for p in (p0, p0 + 1, p0 + 2)])
    close(got, want, tol)


# ------------------------------------------------------------------------------------------------ recurrences
SCANS = [  # H, Hk, dk, dv, taps (0: no convolution, constant decays)
    (6, 2, 16, 24, 4), (3, 3, 24, 16, 0), (4, 1, 33, 20, 3), (2, 2, 64, 72, 0), (2, 1, 128, 64, 2), (5, 5, 40, 100, 1),
    (2, 1, 256, 48, 6), (2, 2, 128, 130, 0), (1, 1, 300, 8, 4), (3, 1, 7, 5, 0)]


def scan_layout(H, Hk, dk, dv, taps):
    if not taps:
        return ops.ScanLayout(rows=2 * Hk * dk + 2 * H * dv, q=0, k=Hk * dk, v=2 * Hk * dk, gate=2 * Hk * dk + H * dv, Hk=Hk,
                              H=H, dk=dk, dv=dv)
    inner, n = H * dv, Hk * dk
    return ops.ScanLayout(rows=2 * inner + 2 * n + H, q=2 * inner + n, k=2 * inner, v=inner, gate=0, Hk=Hk, H=H, dk=dk, dv=dv,
                          taps=taps, conv=inner, channels=inner + 2 * n, dt=2 * inner + 2 * n)


@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("H,Hk,dk,dv,taps", SCANS)
def test_decayed_scan(device, dtype, tol, H, Hk, dk, dv, taps):
    """Convolution, step sizes, decays and the recurrence: prompts by chunks, short portions token by token, state and window
    carried between them in reused slots; one strong and one vanishing decay. The state is compared at fp32 precision
    whatever the storage type: nothing between the activations and the state may be rounded to 16 bits."""
    la = scan_layout(H, Hk, dk, dv, taps)
    lens, rep = (150, 70, 40), H // Hk
    proj = [rnd(n, la.rows, seed=i).to(dtype) for i, n in enumerate(lens)]
    kw, wkw = {}, {}
    if taps:
        C = la.channels
        kw = {"conv_w": rnd(C, taps, seed=5, scale=0.5), "conv_b": rnd(C, seed=6, scale=0.3), "a_log": rnd(H, seed=7),
              "dt_bias": rnd(H, seed=8) - 1, "skip": rnd(H, seed=9)}
        kw["a_log"][0] += 2
        kw["a_log"][-1] -= 5
    else:
        kw = {"log_decay": torch.tensor([-3.0] + [-2.0**-i for i in range(1, H)])[:H].contiguous()}
    wkw = {n: t.double() for n, t in kw.items()}

    def whole(x):
        x = x.double()
        y = x.clone()
        if taps:
            y[:, la.conv:la.conv + la.channels] = O.causal_conv(x[:, la.conv:la.conv + la.channels], wkw["conv_w"],
                                                                wkw["conv_b"])
        y = O.silu(y).to(dtype).double()              # activations are kept in the storage type
        part = lambda at, n, w: y[:, at:at + n * w].view(-1, n, w)
        q, k, v = part(la.q, Hk, dk), part(la.k, Hk, dk), part(la.v, H, dv)
        if taps:
            step = O.softplus(x[:, la.dt:la.dt + H] + wkw["dt_bias"])
            decay = torch.exp(-torch.exp(wkw["a_log"]) * step)
        else:
            step, decay = torch.ones(len(x), H).double(), torch.exp(wkw["log_decay"]).expand(len(x), -1)
        o, S = zip(*[O.decayed_scan(q[:, h // rep], k[:, h // rep], v[:, h], decay[:, h], step[:, h]) for h in range(H)])
        o = torch.stack(o, 1)
        if taps:
            o = o + wkw["skip"][:, None] * v
        return o.reshape(-1, H * dv), torch.stack(S)

    want = [whole(x) for x in proj]
    dks = -(-dk // 8) * 8
    state = torch.full((3, H, dv, dks), 7.0, device=device)    # leftovers of an earlier owner
    state[..., dk:] = 0
    conv = torch.full((3, taps - 1, la.channels), 5.0, dtype=dtype, device=device) if taps > 1 else None
    dkw = {n: t.to(device) for n, t in kw.items()}
    at, got, slot = [0, 0, 0], [[], [], []], (2, 0, 1)
    # (sequence, tokens) portions per step; singles of started sequences first
    for step in ([(0, 100), (1, 3), (2, 17)], [(1, 1), (0, 2), (2, 16)], [(0, 1), (1, 66)], [(0, 47), (2, 7)]):
        mm, _ = meta([(at[i], n) for i, n in step], device, slots=[slot[i] for i, _ in step])
        o = ops.decayed_scan(torch.cat([proj[i][at[i]:at[i] + n] for i, n in step]).to(device), la, state, mm, conv_state=conv,
                             **dkw)
        row = 0
        for i, n in step:
            got[i].append(o[row:row + n])
            row, at[i] = row + n, at[i] + n
    for i in range(3):
        close(torch.cat(got[i]), want[i][0], tol)
        if dtype == torch.float32:
            close(state[slot[i], ..., :dk].transpose(1, 2), want[i][1], 2e-5)
        if taps > 1:
            assert torch.equal(conv[slot[i]].cpu(), proj[i][-(taps - 1):, la.conv:la.conv + la.channels])
    assert not state[..., dk:].any()


@GPU
@pytest.mark.parametrize("dk,dv", [(16, 16), (64, 64), (128, 80), (200, 64)])
def test_chunk_state_is_fp32(dk, dv):
    """The chunked state against fp64, to fp32 precision, from the activations as the device rounds them."""
    from deepspeedsyclsupport_amd.ops.native import scan_ops
    H, n = 2, 333
    la = scan_layout(H, H, dk, dv, 0)
    proj = rnd(n, la.rows, seed=3).bfloat16()
    ld = torch.tensor([-0.002, -0.3])
    m, _ = meta([(0, n)], "cuda", slots=[0])
    dims = (la.rows, la.q, la.k, la.v, la.Hk, la.H, la.dk, la.dv, la.taps, la.conv, la.channels, la.dt)
    qk, v_act, _ = scan_ops().scan_prepare(proj.cuda(), dims, None, None, None, None, None, m.seq_ids, m.cu_q, m.start_pos,
                                           m.slots)
    state = torch.zeros(1, H, dv, -(-dk // 8) * 8, device="cuda")
    ops.decayed_scan(proj.cuda(), la, state, m, log_decay=ld.cuda())
    for h in range(H):
        k, v = qk[1, h, :, :dk].double().cpu(), v_act[h, :, :dv].double().cpu()
        close(k, O.silu(proj[:, la.k + h * dk:la.k + (h + 1) * dk].double()), 1e-2)
        wt = torch.exp(ld[h].double() * torch.arange(n - 1, -1, -1).double())
        close(state[0, h, :, :dk], (v * wt[:, None]).t() @ k, 1e-6 if h else 3e-6)
