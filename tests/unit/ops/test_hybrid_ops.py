"""Each op of the hybrid decoder alone, against the plain functions of the Vopepel oracle: host versions in fp32, gfx950
kernels in fp32 and bf16."""
import pytest
import torch

from deepspeedsyclsupport_amd.inference.model_implementations.transformer import RaggedMeta
from deepspeedsyclsupport_amd.ops import hybrid_ops as ops

from ..inference.v2 import vopepel_oracle as O

GPU = pytest.mark.gpu
CASES = [pytest.param("cpu", torch.float32, 2e-5, id="host"), pytest.param("cuda", torch.float32, 2e-5, id="fp32", marks=GPU),
         pytest.param("cuda", torch.bfloat16, 2e-2, id="bf16", marks=GPU)]


@pytest.fixture(autouse=True)
def _one_thread():
    n = torch.get_num_threads()
    torch.set_num_threads(1)
    yield
    torch.set_num_threads(n)


def rnd(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * scale


def close(got, want, tol):
    got, want = got.double().cpu(), want.double()
    assert got.shape == want.shape
    assert (got - want).abs().max() <= tol * max(1.0, want.abs().max().item())


def meta(portions, device, block=8, slots=None):
    """Ragged batch of (start, new tokens) portions over scattered pages; decodes (one new token) must come first."""
    nb = [-(-(s + n) // block) for s, n in portions]
    ids = torch.randperm(sum(nb) + 3, generator=torch.Generator().manual_seed(1)).tolist()
    blocks = []
    for n in nb:
        blocks.append([ids.pop() for _ in range(n)])
    n_dec = sum(1 for s, n in portions if n == 1 and s > 0)
    return RaggedMeta.build([s for s, _ in portions], [n for _, n in portions], blocks, n_dec, block, device,
                            slots), sum(nb) + 3


@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("S,W", [(1, 64), (4, 132), (3, 37), (2, 4096), (8, 40)])
def test_stream_norm(device, dtype, tol, S, W):
    T, m, eps = 9, 0.6, 1e-4
    mix, out, in_, w = rnd(S, S, seed=1), rnd(S, seed=2), rnd(S, seed=3), 1 + rnd(W, seed=4, scale=0.2)
    embed, ids = rnd(11, W, seed=5).to(dtype), torch.tensor([3, 0, 10, 7, 7, 1, 2, 9, 4], dtype=torch.int32)
    y = rnd(T, W, seed=6).to(dtype)
    xs = embed.double()[ids.long()][None].repeat(S, 1, 1)

    def norm(xs, weights):
        return O.layer_norm(sum(weights[s] * xs[s] for s in range(S)), w.double(), eps)

    d = [t.to(device) for t in (mix, out, in_, w)]
    x = torch.full((T, S, W), float("nan"), device=device)
    h = ops.stream_norm(x, None, None, None, 1.0, d[2], d[3], eps, ids=ids.to(device), embed=embed.to(device))
    assert h.dtype == dtype
    close(h, norm(xs, in_.double()), tol)
    h = ops.stream_norm(x, y.to(device), d[0], d[1], m, d[2], d[3], eps)
    xs = O.stream_mix(xs, y.double(), mix.double(), out.double(), m)
    close(x, xs.transpose(0, 1), 1e-5)      # the streams stay fp32
    close(h, norm(xs, in_.double()), tol)
    rows = torch.tensor([8, 2, 2], dtype=torch.int32, device=device)
    before = x.clone()
    h = ops.stream_norm(x, y.to(device), d[0], d[1], m, None, d[3], eps, rows=rows)
    assert torch.equal(x, before)
    xs = O.stream_mix(xs, y.double(), mix.double(), out.double(), m)
    close(h, norm(xs, torch.ones(S).double())[[8, 2, 2]], tol)


@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("F", [64, 45])
def test_clamped_glu(device, dtype, tol, F):
    gu = rnd(7, 2 * F, scale=2.0).to(dtype)
    for limit in (0.4, 1.0, 7.0):
        close(ops.clamped_glu(gu.to(device), limit), O.clamped_glu(gu[:, :F].double(), gu[:, F:].double(), limit), tol)


@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("H,G,dk,dv", [(4, 2, 32, 16), (6, 6, 20, 36), (12, 1, 64, 128), (2, 1, 136, 24)])
@pytest.mark.parametrize("chunk,window,cap", [(0, 0, 0.0), (13, 0, 5.0), (0, 9, 0.0), (16, 11, 40.0)])
def test_attention(device, dtype, tol, H, G, dk, dv, chunk, window, cap):
    """Epilogue (head norms, value mixing, cache append) and attention over scattered pages: two decodes, a fresh prompt
    and a continued portion in one batch."""
    eps, lam, scale = 1e-5, 0.3, 0.4
    lens = (30, 17, 40, 25)
    qw, kw = 1 + rnd(dk, seed=1, scale=0.3), 1 + rnd(dk, seed=2, scale=0.3)
    N = (H + G) * dk + G * dv
    qkv = [rnd(n, N, seed=10 + i).to(dtype) for i, n in enumerate(lens)]
    vf = [rnd(n, G * dv, seed=20 + i).to(dtype) for i, n in enumerate(lens)]
    m, nb = meta([(0, n) for n in lens], device)
    kc = torch.zeros(nb, G, 8, dk, dtype=dtype, device=device)
    vc = torch.zeros(nb, G, 8, dv, dtype=dtype, device=device)
    lamt = torch.tensor([lam], device=device)

    def run(rows, mm):
        q = ops.qk_norm_append(torch.cat([qkv[i][a:b] for i, a, b in rows]).to(device), qw.to(device), kw.to(device), eps,
                               torch.cat([vf[i][a:b] for i, a, b in rows]).to(device), lamt, mm.pos_ids, mm.seq_ids,
                               mm.block_tables, kc, vc, H)
        return ops.ragged_attention(q, kc, vc, mm, scale, cap, window, chunk)

    # first everything but the last portions, then the batch under test
    portions = [(29, 1), (16, 1), (0, 40), (8, 17)]
    run([(0, 0, 29), (1, 0, 16), (3, 0, 8)], _sub(m, [0, 1, 3], [(0, 29), (0, 16), (0, 8)], device))
    got = run([(i, s, s + n) for i, (s, n) in enumerate(portions)], _sub(m, range(4), portions, device))
    want = []
    for i, (s, n) in enumerate(portions):
        x = qkv[i].double()
        q = O.head_rms_norm(x[:, :H * dk].view(-1, H, dk), qw.double(), eps)
        k = O.head_rms_norm(x[:, H * dk:(H + G) * dk].view(-1, G, dk), kw.double(), eps)
        v = ((1 - lam) * x[:, (H + G) * dk:] + lam * vf[i].double()).view(-1, G, dv)
        o = torch.stack([_attend(q[:, h], k[:, h // (H // G)], v[:, h // (H // G)], scale, cap, chunk, window)
                         for h in range(H)], 1)
        want.append(o[s:s + n])
    close(got, torch.cat(want), tol)


def _attend(q, k, v, scale, cap, chunk, window):
    if not window:
        return O.softmax_attention(q, k, v, scale, cap, chunk)
    return torch.cat([O.softmax_attention(q[lo:i + 1], k[lo:i + 1], v[lo:i + 1], scale, cap, 0)[-1:] for i in range(len(q))
                      for lo in [max(i - window + 1, (i // chunk) * chunk if chunk else 0)]])


def _sub(m, seqs, portions, device):
    bt = m.block_tables.cpu().tolist()
    n_dec = sum(1 for s, n in portions if n == 1 and s > 0)
    return RaggedMeta.build([s for s, _ in portions], [n for _, n in portions], [bt[i] for i in seqs], n_dec, m.block_size,
                            device)


@pytest.mark.parametrize("device,dtype,tol", CASES)
@pytest.mark.parametrize("Hk,rep,dk,dv,taps", [(2, 3, 16, 24, 4), (1, 1, 33, 20, 3), (2, 1, 128, 128, 2), (1, 2, 72, 7, 1),
                                               (1, 1, 256, 200, 6)])
def test_delta_rule(device, dtype, tol, Hk, rep, dk, dv, taps):
    """Convolutions, unit norms, decays, recurrence, head norm and gate; prompts by chunks, short portions token by token,
    state and window carried between them in reused slots; one strong and one vanishing decay."""
    H, eps = Hk * rep, 1e-5
    C, T = 2 * Hk * dk + H * dv, (150, 70, 40)
    NP = C + H * dv + 2 * H
    proj = [rnd(n, NP, seed=i).to(dtype) for i, n in enumerate(T)]
    cw, a_log, dtb, nw = rnd(C, taps, seed=5, scale=0.5), rnd(H, seed=6), rnd(H, seed=7) - 1, 1 + rnd(dv, seed=8, scale=0.2)
    a_log[0] += 2
    a_log[-1] -= 4

    def whole(x):
        x = x.double()
        y = O.silu(O.causal_conv(x[:, :C], cw.double()))
        q = O.unit(y[:, :Hk * dk].view(-1, Hk, dk)) * dk**-0.5
        k = O.unit(y[:, Hk * dk:2 * Hk * dk].view(-1, Hk, dk))
        v = y[:, 2 * Hk * dk:].view(-1, H, dv)
        gate, b, a = x[:, C:C + H * dv].view(-1, H, dv), x[:, C + H * dv:C + H * dv + H], x[:, C + H * dv + H:]
        g = torch.exp(-torch.exp(a_log.double()) * O.softplus(a + dtb.double()))
        o = torch.stack([O.delta_rule(q[:, h // rep], k[:, h // rep], v[:, h], torch.sigmoid(b[:, h]), g[:, h])[0]
                         for h in range(H)], 1)
        return (O.head_rms_norm(o, nw.double(), eps) * O.silu(gate)).reshape(-1, H * dv)

    want = [whole(x) for x in proj]
    state = torch.zeros(3, H, dv, -(-dk // 4) * 4, device=device)
    state[..., :dk] = 7.0                      # leftovers of an earlier owner
    conv = torch.full((3, taps - 1, C), 5.0, dtype=dtype, device=device)
    at, got = [0, 0, 0], [[], [], []]
    # (sequence, tokens) portions per step; singles of started sequences first
    for step in ([(0, 100), (1, 3), (2, 17)], [(1, 1), (0, 2), (2, 16)], [(0, 1), (1, 66)], [(0, 47), (2, 7)]):
        mm, _ = meta([(at[i], n) for i, n in step], device, slots=[(2, 0, 1)[i] for i, _ in step])
        o = ops.delta_rule(torch.cat([proj[i][at[i]:at[i] + n] for i, n in step]).to(device), cw.to(device), a_log.to(device),
                           dtb.to(device), nw.to(device), eps, state, conv, mm, Hk, H, dk, dv)
        row = 0
        for i, n in step:
            got[i].append(o[row:row + n])
            row, at[i] = row + n, at[i] + n
    for i in range(3):
        close(torch.cat(got[i]), want[i], tol)


@GPU
@pytest.mark.parametrize("rows", [1, 2, 5, 16])
@pytest.mark.parametrize("N,K", [(96, 64), (513, 320), (90, 256), (1024, 2048)])
def test_decode_products(rows, N, K):
    from deepspeedsyclsupport_amd.ops.bf16_gemv import Bf16Weight
    x, w = rnd(rows, K).bfloat16().cuda(), rnd(N, K, seed=1, scale=K**-0.5).bfloat16().cuda()
    want = x.double().cpu() @ w.double().cpu().t()
    close(ops.linear(x, w), want, 1e-2)
    close(ops.linear(x, w, Bf16Weight(w)), want, 1e-2)
    if N % 2 == 0:
        glu = O.clamped_glu(want[:, :N // 2], want[:, N // 2:], 0.7)
        close(ops.glu_linear(x, w, None, 0.7), glu, 1e-2)
        close(ops.glu_linear(x, w, Bf16Weight(w), 0.7), glu, 1e-2)
        close(ops.linear(x, w, Bf16Weight(w)), want, 1e-2)   # the gated finalize leaves the sums cleared
