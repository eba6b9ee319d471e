"""Plain-PyTorch fp32 reference implementations.

Used (1) as the numerics oracle in tests of the HIP kernels and (2) for host (CPU) tensors on the gloo plumbing
path. Device tensors never come here (see `ops/native.py`).
"""
import math

import torch
import torch.nn.functional as F


def adam_update(p, m, v, g, lr, beta1, beta2, eps, wd, step, bias_correction=True, adamw=True, grad_scale=1.0,
                lp=None):
    gf = g.float() * grad_scale
    pf = p.float()
    if not adamw and wd != 0:
        gf = gf + wd * pf
    mf = m.float().mul_(beta1).add_(gf, alpha=1 - beta1)
    vf = v.float().mul_(beta2).addcmul_(gf, gf, value=1 - beta2)
    bc1 = 1 - beta1**step if bias_correction else 1.0
    bc2 = 1 - beta2**step if bias_correction else 1.0
    denom = vf.sqrt() / math.sqrt(bc2) + eps
    upd = (mf / bc1) / denom
    if adamw and wd != 0:
        upd = upd + wd * pf
    pf = pf - lr * upd
    p.copy_(pf)
    m.copy_(mf)
    v.copy_(vf)
    if lp is not None:
        lp.copy_(pf)


def lion_update(p, m, g, lr, beta1, beta2, wd, grad_scale=1.0, lp=None):
    gf = g.float() * grad_scale
    pf = p.float()
    mf = m.float()
    c = beta1 * mf + (1 - beta1) * gf
    pf = pf * (1 - lr * wd) - lr * torch.sign(c)
    mf = beta2 * mf + (1 - beta2) * gf
    p.copy_(pf)
    m.copy_(mf)
    if lp is not None:
        lp.copy_(pf)


def adagrad_update(p, s, g, lr, eps, wd, grad_scale=1.0, lp=None):
    gf = g.float() * grad_scale
    pf = p.float()
    if wd != 0:
        gf = gf + wd * pf
    sf = s.float() + gf * gf
    pf = pf - lr * gf / (sf.sqrt() + eps)
    p.copy_(pf)
    s.copy_(sf)
    if lp is not None:
        lp.copy_(pf)


def lamb_update(p, m, v, g, lr, beta1, beta2, eps, wd, step, bias_correction=True, grad_scale=1.0, max_coeff=10.0,
                min_coeff=0.01, lp=None):
    gf = g.float() * grad_scale
    pf = p.float()
    mf = m.float().mul_(beta1).add_(gf, alpha=1 - beta1)
    vf = v.float().mul_(beta2).addcmul_(gf, gf, value=1 - beta2)
    bc1 = 1 - beta1**step if bias_correction else 1.0
    bc2 = 1 - beta2**step if bias_correction else 1.0
    u = (mf / bc1) / ((vf / bc2).sqrt() + eps) + wd * pf
    wn, un = pf.norm(), u.norm()
    trust = (wn / un) if (wn > 0 and un > 0) else torch.tensor(1.0)
    trust = float(min(max(float(trust), min_coeff), max_coeff))
    pf = pf - lr * trust * u
    p.copy_(pf)
    m.copy_(mf)
    v.copy_(vf)
    if lp is not None:
        lp.copy_(pf)
    return trust


def rms_norm(x, w, eps, residual=None):
    h = x.float() + residual.float() if residual is not None else x.float()
    y = h * torch.rsqrt(h.pow(2).mean(-1, keepdim=True) + eps) * w.float()
    return y.to(x.dtype), (h.to(x.dtype) if residual is not None else None)


def layer_norm(x, g, b, eps, residual=None):
    h = x.float() + residual.float() if residual is not None else x.float()
    y = F.layer_norm(h, (h.shape[-1], ), g.float(), b.float(), eps)
    return y.to(x.dtype), (h.to(x.dtype) if residual is not None else None)


ACTS = {0: F.silu, 1: lambda x: F.gelu(x, approximate="tanh"), 2: F.gelu, 3: F.relu, 4: lambda x: x}


def gated_act(gu, act=0):
    g, u = gu.float().chunk(2, dim=-1)
    return (ACTS[act](g) * u).to(gu.dtype)


def rope_tables(max_pos, rot, base=10000.0, scaling=None, device=None):
    inv = 1.0 / (base**(torch.arange(0, rot, 2, dtype=torch.float64) / rot))
    t = torch.arange(max_pos, dtype=torch.float64)
    if scaling:
        t = t / scaling
    f = torch.outer(t, inv)
    return f.cos().float().to(device), f.sin().float().to(device)


def apply_rope_half(x, cos, sin, pos):
    """x [B, S, H, D] (rotate_half on the first 2*cos.shape[-1] dims); pos [S] or [B,S] long."""
    rot = cos.shape[-1] * 2
    c = cos[pos].float()
    s = sin[pos].float()
    if c.dim() == 2:
        c, s = c[None, :, None, :], s[None, :, None, :]
    else:
        c, s = c[:, :, None, :], s[:, :, None, :]
    xf = x.float()
    x1, x2, rest = xf[..., :rot // 2], xf[..., rot // 2:rot], xf[..., rot:]
    o1 = x1 * c - x2 * s
    o2 = x2 * c + x1 * s
    return torch.cat([o1, o2, rest], dim=-1).to(x.dtype)


def cross_entropy(logits, labels, ignore_index=-100, smoothing=0.0):
    return F.cross_entropy(logits.float(), labels, ignore_index=ignore_index, reduction="none",
                           label_smoothing=smoothing)


# ------------------------------------------------------------------------------------------------ hybrid decoder
def stream_norm(x, y, mix, out, m, in_, w, eps, ids=None, embed=None, rows=None):
    """Multi-stream residual update (in place on x [T, S, W]) + layer norm of the streams' weighted sum."""
    src = y if y is not None else embed
    if y is not None:
        xn = torch.einsum("st,nsw->ntw", mix, x) + m * out[None, :, None] * y.float().view(x.shape[0], 1, -1)
    else:
        xn = embed.float()[ids.long()][:, None].expand(-1, x.shape[1], -1)
    if rows is not None:
        xn = xn[rows.long()]
    else:
        x.copy_(xn)
    u = (xn if in_ is None else xn * in_[None, :, None]).sum(1)
    d = u - u.mean(-1, keepdim=True)
    return (d * torch.rsqrt(d.pow(2).mean(-1, keepdim=True) + eps) * w).to(src.dtype)


def clamped_glu(gu, limit, alpha, shift):
    g, u = gu.float().chunk(2, -1)
    g = g.clamp(max=limit)
    return (g * torch.sigmoid(alpha * g) * (u.clamp(-limit, limit) + shift)).to(gu.dtype)


def qk_norm_append(qkv, qw, kw, eps, vfirst, lam, pos, seq_ids, block_table, kc, vc, H, cs=None):
    G, BS, dk, dv = kc.shape[1], kc.shape[2], kc.shape[3], vc.shape[3]
    T = qkv.shape[0]
    q, k, v = qkv.float().split([H * dk, G * dk, G * dv], -1)
    q, k, v = _turn_neighbours(q.view(T, H, dk), cs), _turn_neighbours(k.view(T, G, dk), cs), v.reshape(T, G, dv)
    q = q * torch.rsqrt(q.pow(2).mean(-1, keepdim=True) + eps) * (1.0 if qw is None else qw)
    k = k * torch.rsqrt(k.pow(2).mean(-1, keepdim=True) + eps) * (1.0 if kw is None else kw)
    if vfirst is not None:
        v = (1 - lam) * v + lam * vfirst.float().view(T, G, dv)
    slot = pos.long()
    blk = block_table.long()[seq_ids.long(), slot // BS]
    kc[blk, :, slot % BS] = k.to(kc.dtype)
    vc[blk, :, slot % BS] = v.to(vc.dtype)
    return q.to(qkv.dtype)


def rope_table(pos, freq, mult):
    a = pos.double()[:, None] * freq.double()
    return torch.stack([a.cos(), a.sin()], -1).float() * mult


def _turn_pairs(x, cs):
    """x [T, heads, d]: pairs (i, i + half) turned by cs [T, half, 2]."""
    if cs is None:
        return x
    h, (c, s) = cs.shape[1], cs[:, None].unbind(-1)
    u, v = x[..., :h], x[..., h:2 * h]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * h:]], -1)


def _turn_neighbours(x, cs):
    """x [T, heads, d]: pairs (2 i, 2 i + 1) turned by cs [T, half, 2]."""
    if cs is None:
        return x
    h, (c, s) = cs.shape[1], cs[:, None].unbind(-1)
    u, v = x[..., 0:2 * h:2], x[..., 1:2 * h:2]
    return torch.cat([torch.stack([u * c - v * s, v * c + u * s], -1).flatten(-2), x[..., 2 * h:]], -1)


def qk_rope_append(qkv, bias, qw, kw, eps, cs, v_mult, pos, seq_ids, block_table, kc, vc, H):
    G, BS, dk, dv = kc.shape[1], kc.shape[2], kc.shape[3], vc.shape[3]
    T = qkv.shape[0]
    q, k, v = (qkv.float() if bias is None else qkv.float() + bias).split([H * dk, G * dk, G * dv], -1)
    q, k = (x if w is None else _rms(x, eps) * w for x, w in ((q, qw), (k, kw)))
    q, k, v = _turn_pairs(q.view(T, H, dk), cs), _turn_pairs(k.view(T, G, dk), cs), v.reshape(T, G, dv) * v_mult
    slot = pos.long()
    blk = block_table.long()[seq_ids.long(), slot // BS]
    kc[blk, :, slot % BS] = k.to(kc.dtype)
    vc[blk, :, slot % BS] = v.to(vc.dtype)
    return q.to(qkv.dtype)


def paged_attention(q, kc, vc, block_table, pos, seq_ids, scale, softcap, window, chunk, sink=None, gate=None):
    """q [T, H, dk] at absolute positions -> [T, H, dv]; visible keys [lo(pos), pos] (window / chunk start / 0). `gate` [T, H]:
    heads come out times its sigmoid."""
    G, BS = kc.shape[1], kc.shape[2]
    out = q.new_empty(q.shape[0], q.shape[1], vc.shape[3])
    for t in range(q.shape[0]):
        p = int(pos[t])
        lo = max(p // chunk * chunk if chunk else 0, p - window + 1 if window else 0)
        j = torch.arange(lo, p + 1)
        blk = block_table[int(seq_ids[t])].long()[j // BS]
        k, v = kc[blk, :, j % BS].float(), vc[blk, :, j % BS].float()         # [n, G, d]
        qq = q[t].float().view(G, q.shape[1] // G, -1)
        s = torch.einsum("grd,ngd->grn", qq, k) * scale
        if softcap:
            s = softcap * torch.tanh(s / softcap)
        if sink is not None:
            p = torch.cat([s, sink.view(G, -1, 1)], -1).softmax(-1)[..., :-1]
        else:
            p = s.softmax(-1)
        o = torch.einsum("grn,ngd->grd", p, v).reshape(q.shape[1], -1)
        out[t] = (o if gate is None else o * torch.sigmoid(gate[t].float())[:, None]).to(q.dtype)
    return out


def delta_prepare(proj, conv_w, conv_state, a_log, dt_bias, seq_ids, cu, start, slots, Hk, H, dk, dv):
    T, taps = proj.shape[0], conv_w.shape[-1]
    C = 2 * Hk * dk + H * dv
    x = torch.empty(T, C)
    for i in range(start.numel()):
        a, b, slot = int(cu[i]), int(cu[i + 1]), int(slots[i])
        old = conv_state[slot].float() if int(start[i]) else torch.zeros(taps - 1, C)
        seq = torch.cat([old, proj[a:b, :C].float()])
        x[a:b] = sum(seq[j:j + b - a] * conv_w[:, j] for j in range(taps))
    x = F.silu(x)
    q, k, v = x.split([Hk * dk, Hk * dk, H * dv], -1)
    q, k = q.view(T, Hk, dk), k.view(T, Hk, dk)
    q = q * torch.rsqrt(q.pow(2).sum(-1, keepdim=True) + 1e-6) * dk**-0.5
    k = k * torch.rsqrt(k.pow(2).sum(-1, keepdim=True) + 1e-6)
    b, a = proj[:, C + H * dv:].float().split(H, -1)
    glog = -a_log.exp() * F.softplus(a + dt_bias)
    return torch.stack([q, k], 1), v.view(T, H, dv).to(proj.dtype), torch.stack([glog, b.sigmoid()], 1)


def delta_recur(qk, v, gb, proj, norm_w, eps, state, conv_state, seqs, cu, start, slots, out, dk):
    T, H, dv = v.shape
    Hk = qk.shape[2]
    C, taps = conv_state.shape[2], conv_state.shape[1] + 1
    out = out.view(T, H, dv)
    rep = H // Hk
    for i in seqs.tolist():
        a, b, slot = int(cu[i]), int(cu[i + 1]), int(slots[i])
        S = state[slot, ..., :dk].transpose(1, 2).clone() if int(start[i]) else torch.zeros(H, dk, dv)
        for t in range(a, b):
            q, k = qk[t].repeat_interleave(rep, 1)
            S = S * gb[t, 0].exp()[:, None, None]
            u = gb[t, 1][:, None] * (v[t].float() - (S * k[:, :, None]).sum(1))
            S = S + k[:, :, None] * u[:, None]
            o = (S * q[:, :, None]).sum(1)
            o = o * torch.rsqrt(o.pow(2).mean(-1, keepdim=True) + eps) * norm_w
            out[t] = (o * F.silu(proj[t, C:C + H * dv].float().view(H, dv))).to(out.dtype)
        state[slot, ..., :dk] = S.transpose(1, 2)
        if taps > 1:
            old = conv_state[slot] if int(start[i]) else torch.zeros_like(conv_state[slot])
            conv_state[slot] = torch.cat([old, proj[a:b, :C]])[-(taps - 1):].clone()


def delta_chunk(qk, v, gb, proj, norm_w, eps, state, conv_state, seqs, work, cu, start, slots, out, dk):
    """Long portions: the same recurrence (the device splits it into chunks)."""
    delta_recur(qk, v, gb, proj, norm_w, eps, state, conv_state, seqs[:, 0], cu, start, slots, out, dk)


# ---------------------------------------------------------------- latent attention, decayed scans, post-norm residual
def _rms(x, eps):
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def post_norm(x, y, w, eps, ids, embed, rows, final_w, mult):
    if y is None:
        x.copy_(embed.float()[ids.long()])
        return x.to(embed.dtype)
    s = x + _rms(y.float().view(x.shape), eps) * w
    if rows is not None:
        return (_rms(s[rows.long()], eps) * final_w * mult).to(y.dtype)
    x.copy_(s)
    return x.to(y.dtype)


def gelu_erf(x):
    return F.gelu(x.float()).to(x.dtype)


def token_gate(g, ids, table, first):
    e = table[ids.long(), first:first + g.shape[-1]].float()
    return (F.gelu(g.float(), approximate="tanh") * e).to(g.dtype)


def gated_norm(y, proj, gate, w, parts, eps, mode, out=None):
    T, C = y.shape
    g, v = proj[:, gate:gate + C].float(), y.float()
    if mode == 1:
        v = v * F.silu(g)
    v = _rms(v.view(T, parts, C // parts), eps).view(T, C) * (1.0 if w is None else w)
    v = (v * torch.sigmoid(g) if mode == 0 else v * F.silu(g) if mode == 2 else v).to(y.dtype)
    return v if out is None else out.copy_(v)


def _turn(x, freq, mult, pos):
    """Rotate-half on the first 2 len(freq) columns of x [T, .., r] at positions pos [T], cosine and sine times `mult`."""
    h = freq.numel()
    a = (pos.double()[:, None] * freq.double()).view(-1, *[1] * (x.dim() - 2), h)
    c, s = a.cos().float() * mult, a.sin().float() * mult
    u, v = x[..., :h], x[..., h:2 * h]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * h:]], -1)


def latent_prepare(down, qw, kvw, eps, freq, mult, pos, seq_ids, block_table, lat, q_rank):
    R, BS = kvw.numel(), lat.shape[2]
    d = down.float()
    rows = torch.cat([_rms(d[:, q_rank:q_rank + R], eps) * kvw, _turn(d[:, q_rank + R:], freq, mult, pos)], -1)
    slot = pos.long()
    lat[block_table.long()[seq_ids.long(), slot // BS], 0, slot % BS] = rows.to(lat.dtype)
    return (_rms(d[:, :q_rank], eps) * qw).to(down.dtype) if q_rank else None


def latent_attention(q, lat, ukv, freq, mult, sink, block_table, pos, seq_ids, scale, d, e, window=0):
    T, H = q.shape[:2]
    R, BS = ukv.shape[1], lat.shape[2]
    uk, uv = ukv.float().split([H * d, H * e])
    q = torch.cat([q[..., :d].float(), _turn(q[..., d:].float(), freq, mult, pos)], -1)
    out = q.new_empty(T, H, e, dtype=ukv.dtype)
    for s in seq_ids.unique().tolist():
        rows = (seq_ids == s).nonzero().view(-1)
        j = torch.arange(int(pos[rows].max()) + 1)
        c = lat[block_table[s].long()[j // BS], 0, j % BS].float()
        k = torch.cat([(c[:, :R] @ uk.t()).view(-1, H, d), c[:, None, R:].expand(-1, H, -1)], -1)
        v = (c[:, :R] @ uv.t()).view(-1, H, e)
        sc = torch.einsum("thd,jhd->htj", q[rows], k) * scale
        hidden = j > pos[rows][:, None]
        if window:
            hidden |= j <= pos[rows][:, None] - window
        sc = sc.masked_fill(hidden, float("-inf"))
        if sink is None:
            p = sc.softmax(-1)
        else:
            p = torch.cat([sc, sink[:, None, None].expand(-1, rows.numel(), 1)], -1).softmax(-1)[..., :-1]
        out[rows] = torch.einsum("htj,jhe->the", p, v).to(out.dtype)
    return out


def _scan_dims(dims):
    return dict(zip(("rows", "q", "k", "v", "Hk", "H", "dk", "dv", "taps", "conv", "channels", "dt"), dims))


def scan_prepare(proj, dims, conv_w, conv_b, conv_state, a_log, dt_bias, seq_ids, cu, start, slots):
    D = _scan_dims(dims)
    T, x = proj.shape[0], proj.float().clone()
    if conv_w is not None:
        c0, C, taps = D["conv"], D["channels"], D["taps"]
        for i in range(start.numel()):
            a, b = int(cu[i]), int(cu[i + 1])
            old = conv_state[int(slots[i])].float() if int(start[i]) and taps > 1 else torch.zeros(taps - 1, C)
            seq = torch.cat([old, proj[a:b, c0:c0 + C].float()])
            x[a:b, c0:c0 + C] = sum(seq[j:j + b - a] * conv_w[:, j] for j in range(taps)) + conv_b
    part = lambda at, n, w: F.silu(x[:, at:at + n * w]).view(T, n, w).to(proj.dtype)
    qk = torch.stack([part(D["q"], D["Hk"], D["dk"]), part(D["k"], D["Hk"], D["dk"])], 1)
    gb = None
    if D["dt"] >= 0:
        b = F.softplus(proj[:, D["dt"]:D["dt"] + D["H"]].float() + dt_bias)
        gb = torch.stack([-a_log.exp() * b, b], 1)
    return qk, part(D["v"], D["H"], D["dv"]), gb


def scan_split(proj, dims, cs):
    D = _scan_dims(dims)
    part = lambda at, n, w: proj[:, at:at + n * w].reshape(-1, n, w)
    q, k = (_turn_pairs(part(D[c], D["Hk"], D["dk"]).float(), cs).to(proj.dtype) for c in "qk")
    return torch.stack([q, k], 1), part(D["v"], D["H"], D["dv"])


def exp_gates(proj, ci, cf, bi, bf, cap, peak, cu, start, slots, longest):
    H = bi.numel()
    i = cap * torch.tanh((proj[:, ci:ci + H].float() + bi) / cap)
    f = F.logsigmoid(cap * torch.tanh((proj[:, cf:cf + H].float() + bf) / cap))
    gb, floors = torch.empty(proj.shape[0], 2, H), torch.empty(proj.shape[0], H)
    for s in range(start.numel()):
        m = peak[int(slots[s])].clone() if int(start[s]) else torch.zeros(H)
        for t in range(int(cu[s]), int(cu[s + 1])):
            new = torch.maximum(f[t] + m, i[t])
            gb[t, 0], gb[t, 1], floors[t], m = f[t] + m - new, (i[t] - new).exp(), (-new).exp(), new
        peak[int(slots[s])] = m
    return gb, floors


def scan_recur(qk, v, gb, log_decay, skip, scale, proj, dims, state, zstate, floors, conv_state, seqs, cu, start, slots, out):
    D = _scan_dims(dims)
    T, H, dk = proj.shape[0], D["H"], D["dk"]
    rep, out = H // D["Hk"], out.view(T, H, D["dv"])
    for i in seqs.tolist():
        a, b, slot, old = int(cu[i]), int(cu[i + 1]), int(slots[i]), int(start[i]) > 0
        S = state[slot, ..., :dk].transpose(1, 2).clone() if old else torch.zeros(H, dk, D["dv"])
        Z = zstate[slot, :, 0, :dk].clone() if zstate is not None and old else torch.zeros(H, dk)
        for t in range(a, b):
            q, k = qk[t].float().repeat_interleave(rep, 1)
            g, step = (gb[t, 0], gb[t, 1]) if gb is not None else (log_decay, torch.ones(H))
            S = S * g.exp()[:, None, None] + (k * step[:, None])[:, :, None] * v[t].float()[:, None]
            o = scale * (S * q[:, :, None]).sum(1)
            if zstate is not None:
                Z = Z * g.exp()[:, None] + k * step[:, None]
                o = o / (torch.maximum((scale * (Z * q).sum(-1)).abs(), floors[t]) + 1e-6)[:, None]
            out[t] = (o if skip is None else o + skip[:, None] * v[t].float()).to(out.dtype)
        state[slot, ..., :dk] = S.transpose(1, 2)
        if zstate is not None:
            zstate[slot, ..., :dk] = Z[:, None]
        if conv_state is not None and conv_state.shape[1]:
            before = conv_state[slot] if old else torch.zeros_like(conv_state[slot])
            new = proj[a:b, D["conv"]:D["conv"] + D["channels"]]
            conv_state[slot] = torch.cat([before, new])[-(D["taps"] - 1):].clone()


def scan_chunk(qk, v, gb, log_decay, skip, scale, proj, dims, state, zstate, floors, conv_state, seqs, cu, start, slots, out):
    """Long portions: the same recurrence (the device splits it into chunks)."""
    scan_recur(qk, v, gb, log_decay, skip, scale, proj, dims, state, zstate, floors, conv_state, seqs[:, 0], cu, start, slots,
               out)


# ---------------------------------------------------------------- pre-norm residual, experts with grouped routing
def expert_sum(y, w, rows, base=None):
    T, K = w.shape
    e = y.float()[rows.long().view(-1)] if rows is not None else y.float()
    s = (e.view(T, K, -1) * w[..., None]).sum(1)
    return (s if base is None else s + base.float()).to(y.dtype)


def pre_norm(x, y, yw, yrow, base, w, eps, ids, embed, mult, rows, post_w, gate, gate_b):
    norm = lambda s: s if w is None else _rms(s, eps) * w
    if y is None:
        x.copy_(embed.float()[ids.long()] * mult)
        return norm(x).to(embed.dtype)
    add = y.float() if yw is None else expert_sum(y.float(), yw, yrow, base)
    if gate is not None:
        add = add * torch.sigmoid(gate.float() + gate_b)
    if post_w is not None:
        add = _rms(add, eps) * post_w
    s = x + add
    if rows is not None:
        return norm(s[rows.long()]).to(y.dtype)
    x.copy_(s)
    return norm(s).to(y.dtype)


def route(h, router, k, groups, keep, score=0, best=1, scale=1.0):
    z = h.float() @ router.float().t()
    s = torch.sigmoid(z) if score else z.softmax(-1)
    T, E = s.shape
    per = E // groups
    top = s.view(T, groups, per).topk(min(best, per), -1).values.sum(-1).topk(keep, -1).indices
    open_ = torch.zeros(T, groups, dtype=torch.bool).scatter_(1, top, True).repeat_interleave(per, 1)
    w, e = s.masked_fill(~open_, -1.0).topk(k, -1)
    return e.to(torch.int32), w / (w.sum(-1, keepdim=True) + 1e-20) * scale


def row_act(x, act):
    if act == 1:
        g, u = x.float().chunk(2, -1)
        return (F.silu(g) * u).to(x.dtype)
    return x.float().clamp(min=0).square().to(x.dtype) if act == 2 else x


def expert_gemm(x, w, experts, div, act):
    out = x.new_empty(experts.numel(), w.shape[1] // (2 if act == 1 else 1))
    e = experts.view(-1).long()
    for i in e.unique().tolist():
        r = (e == i).nonzero().view(-1)
        out[r] = row_act(F.linear(x[r // div], w[i]), act)
    return out


# ---------------------------------------------------------------- recurrences with a decay per channel and state
def causal_conv(x, w, b, conv_state, cu, start, slots):
    T, C = x.shape
    taps, y = w.shape[1], torch.empty(T, C)
    for i in range(start.numel()):
        p, q = int(cu[i]), int(cu[i + 1])
        old = conv_state[int(slots[i])].float() if int(start[i]) and taps > 1 else torch.zeros(taps - 1, C)
        seq = torch.cat([old, x[p:q].float()])
        y[p:q] = sum(seq[j:j + q - p] * w[:, j] for j in range(taps)) + b
    return F.silu(y).to(x.dtype)


def selective_scan(x, dt, bc, z, dt_bias, decay, skip, state, conv_x, conv_state, seqs, cu, start, slots, steps, out):
    C, N = decay.shape
    step = F.softplus(dt.float() + dt_bias, threshold=60)
    for i in (seqs if steps else seqs[:, 0]).tolist():
        p, q, slot, old = int(cu[i]), int(cu[i + 1]), int(slots[i]), int(start[i]) > 0
        S = state[slot, :, :N].clone() if old else torch.zeros(C, N)
        for t in range(p, q):
            xt, B, Ct = x[t].float(), bc[t, :N].float(), bc[t, N:2 * N].float()
            S = (step[t][:, None] * decay).exp() * S + (step[t] * xt)[:, None] * B
            out[t] = (((S * Ct).sum(-1) + skip * xt) * F.silu(z[t].float())).to(out.dtype)
        state[slot, :, :N] = S
        if conv_state is not None and conv_state.shape[1]:
            before = conv_state[slot] if old else torch.zeros_like(conv_state[slot])
            conv_state[slot] = torch.cat([before, conv_x[p:q]])[-conv_state.shape[1]:].clone()
