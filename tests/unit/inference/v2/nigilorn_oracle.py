"""Plain, slow implementation of the Nigilorn decoder for tests: one whole sequence at a time, one function per mechanism,
written straight from the model's equations in PyTorch on the CPU. It shares no code with the package.

Weights come as a dict of tensors under the checkpoint's names; arithmetic runs in the dtype of `cast` (float64 by
default). Nothing here is cached, paged, batched, absorbed, chunked or fused. Under `Rounded()` the operands and results of
the projections are rounded to bf16: what a model in 16 bits cannot do better than."""
import math

import torch


class Rounded:
    """Context in which `project` works on bf16 operands and results."""
    on = False

    def __enter__(self):
        Rounded.on = True

    def __exit__(self, *exc):
        Rounded.on = False


def project(x, w):
    """W x for every row."""
    if not Rounded.on:
        return x @ w.t()
    return (x.bfloat16().to(w.dtype) @ w.t()).bfloat16().to(w.dtype)


# ------------------------------------------------------------------------------------------------ mechanisms
def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(x):
    return 1 / (1 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    """log(1 + e^x), without overflow."""
    return torch.clamp(x, min=0) + torch.log1p(torch.exp(-x.abs()))


def gelu_tanh(x):
    return 0.5 * x * (1 + torch.tanh(math.sqrt(2 / math.pi) * (x + 0.044715 * x**3)))


def yarn(rot):
    """(frequency of every pair, factor of cosine and sine): pairs that turn often within the original length keep their
    frequency, those that hardly turn are slowed down by the factor, with a linear ramp between."""
    dims, base, sc = rot["dims"], rot["base"], rot["scaling"]

    def pair_of(turns):
        return dims * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo, hi = max(math.floor(pair_of(sc["fast"])), 0), min(math.ceil(pair_of(sc["slow"])), dims - 1)
    out = []
    for i in range(dims // 2):
        f, ramp = base**(-2 * i / dims), min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / sc["factor"] * ramp + f * (1 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1


def rotate(x, rot, first=0):
    """x [n, d]: row i sits at position first + i; neighbours (2 j, 2 j + 1) of the first `dims` elements turn by
    position * frequency_j and grow by the factor."""
    freq, grow = yarn(rot)
    out = x.clone()
    for j, f in enumerate(freq):
        a = torch.arange(first, first + x.shape[0], dtype=torch.float64) * f
        c, s = (grow * torch.cos(a)).to(x.dtype), (grow * torch.sin(a)).to(x.dtype)
        u, v = x[:, 2 * j], x[:, 2 * j + 1]
        out[:, 2 * j], out[:, 2 * j + 1] = u * c - v * s, v * c + u * s
    return out


def window_attention(q, k, v, scale, window):
    """One head: q, k [n, d], v [n, e]. Query i sees itself and the window - 1 keys before it."""
    out = []
    for i in range(q.shape[0]):
        lo = max(i - window + 1, 0)
        out.append(torch.softmax((k[lo:i + 1] @ q[i]) * scale, -1) @ v[lo:i + 1])
    return torch.stack(out)


def causal_conv(x, taps, bias):
    """x [n, C], taps [C, L] (last column: the current token), bias [C] -> [n, C], zeros before the first token."""
    n, L = x.shape[0], taps.shape[1]
    out = bias.expand(n, -1).clone()
    for j in range(L):
        back = L - 1 - j
        if back < n:
            out[back:] += taps[:, j] * x[:n - back]
    return out


def selective_scan(x, dt, A, B, C):
    """x, dt [n, channels], A [channels, N], B, C [n, N]: every channel carries N numbers, each with its own decay."""
    S, out = torch.zeros_like(A), []
    for t in range(x.shape[0]):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        out.append(S @ C[t])
    return torch.stack(out)


def route(z, top, groups, keep, scale):
    """Router logits z [n, E] -> (experts [n, top], weights [n, top]): the best experts of the `keep` best groups by sigmoid (a
    group is as good as its two best members together), weighted by their share of the chosen ones' sum, times `scale`."""
    s = sigmoid(z)
    n, E = s.shape
    per = E // groups
    worth = s.view(n, groups, per).sort(-1, descending=True).values[..., :2].sum(-1)
    allowed = torch.zeros(n, groups, dtype=torch.bool).scatter_(1, worth.topk(keep, -1).indices, True)
    e = s.masked_fill(~allowed.repeat_interleave(per, 1), -1.0).topk(top, -1).indices
    w = s.gather(1, e)
    return e, w / (w.sum(-1, keepdim=True) + 1e-20) * scale


# ------------------------------------------------------------------------------------------------ layers
def mamba_mixer(w, p, mx, h, eps):
    inner, N, R = mx["inner"], mx["state"], mx["dt_rank"]
    x, z = project(h, w[p + "in"]).split(inner, -1)
    x = silu(causal_conv(x, w[p + "conv"], w[p + "conv.b"]))
    dt, B, C = project(x, w[p + "x"]).split([R, N, N], -1)
    dt = softplus(project(dt, w[p + "dt"]) + w[p + "dt.b"])
    y = selective_scan(x, dt, -torch.exp(w[p + "A_log"]), B, C) + w[p + "D"] * x
    return project(y * silu(z), w[p + "o"])


def attention_mixer(w, p, mx, h, eps):
    n, H, G, d, e = h.shape[0], mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q, k, v = (project(h, w[p + c]).view(n, m, -1) for c, m in (("q", H), ("k", G), ("v", G)))
    turn = lambda x: rms(rotate(x, mx["rot"]), eps)
    ks = [turn(k[:, g]) for g in range(G)]
    out = torch.stack([window_attention(turn(q[:, i]), ks[i // (H // G)], v[:, i // (H // G)], mx["scale"], mx["mask"]["size"])
                       for i in range(H)], 1)
    out = out * sigmoid(project(h, w[p + "g"]))[..., None]
    return project(out.reshape(n, H * e), w[p + "o"])


def latent_mixer(w, p, mx, h, eps):
    n, H, d, r, e, R = h.shape[0], mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
    q, down = project(h, w[p + "q"]).view(n, H, d + r), project(h, w[p + "dkv"])
    c = rms(down[:, :R], eps) * w[p + "dkv.norm"]
    kr = rotate(down[:, R:], mx["rot"])
    k, v = project(c, w[p + "uk"]).view(n, H, d), project(c, w[p + "uv"]).view(n, H, e)
    out = [window_attention(torch.cat([q[:, i, :d], rotate(q[:, i, d:], mx["rot"])], -1), torch.cat([k[:, i], kr], -1), v[:, i],
                            mx["scale"], mx["mask"]["size"]) for i in range(H)]
    return project(torch.stack(out, 1).reshape(n, H * e), w[p + "o"])


MIXERS = {"mamba1": mamba_mixer, "attention": attention_mixer, "latent_attention": latent_mixer}


def gated_ff(w, p, h):
    return project(silu(project(h, w[p + "gate"])) * project(h, w[p + "up"]), w[p + "down"])


def relu2_ff(w, p, h):
    return project(torch.clamp(project(h, w[p + "up"]), min=0)**2, w[p + "down"])


def experts(w, p, ml, h):
    r = ml["router"]
    e, wt = route(h @ w[p + "router"].t(), r["top"], r["groups"]["count"], r["groups"]["keep"], r["scale"])
    out = relu2_ff(w, p + "shared.", h)
    for t in range(h.shape[0]):
        for j in range(r["top"]):
            out[t] += wt[t, j] * relu2_ff(w, f"{p}e{int(e[t, j])}.", h[t:t + 1])[0]
    return out


def feed_forward(w, p, ml, h):
    return gated_ff(w, p, h) if ml["kind"] == "dense" else experts(w, p, ml, h)


def sublayer(w, p, q, x, f, eps):
    """x + norm(gate(h) * f(h)) with h the normed x; q: "1" or "2"."""
    h = rms(x, eps) * w[p + "norm" + q]
    g = sigmoid(project(h, w[p + "rg" + q]) + w[p + f"rg{q}.b"])
    return x + rms(g * f(h), eps) * w[p + f"norm{q}b"]


def token_side(w, p, dim, i, x, ids, eps):
    """The layer's own embedding of each token, gated by the residual and added to it."""
    e = w["side.embed"][ids][:, i * dim:(i + 1) * dim]
    y = project(gelu_tanh(project(x, w[p + "side.gate"])) * e, w[p + "side.proj"])
    return x + rms(y, eps) * w[p + "side.norm"]


def forward(cfg, weights, tokens, cast=torch.float64, trace=None):
    """Logits [n, vocab] of one sequence; `trace` (a list) receives the residual after every layer."""
    w = {k: v.to(cast) for k, v in weights.items()}
    eps, ids = cfg["norm"]["eps"], torch.as_tensor(tokens).long()
    x = w["embed"][ids]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = sublayer(w, p, "1", x, lambda h: MIXERS[layer["type"]](w, p + "mix.", layer["mixer"], h, eps), eps)
        if layer.get("mlp"):
            x = sublayer(w, p, "2", x, lambda h: feed_forward(w, p + "mlp.", layer["mlp"], h), eps)
        x = token_side(w, p, cfg["token_side"]["dim"], i, x, ids, eps)
        if trace is not None:
            trace.append(x)
    return project(rms(x, eps) * w["final.norm"], w["head"])


# ------------------------------------------------------------------------------------------------ test models
CODE = 8   # columns of the residual that `decisive` models keep for the router


def random_model(cfg, seed=0, dtype=torch.bfloat16, decisive=False):
    """Random weights for a config. `decisive`: the last `CODE` columns of the residual belong to the router alone (no sublayer
    writes them, the embedding does), with values drawn anew until no token comes near a tie in any layer. Rounding then cannot
    change an expert, so that whole models compare in 16 bits."""
    g = torch.Generator().manual_seed(seed)
    W, w = cfg["width"], {}

    def put(name, shape, std=None, mean=0.0):
        std = std if std is not None else 1 / math.sqrt(shape[-1])
        w[name] = (torch.randn(shape, generator=g) * std + mean).to(dtype)

    put("embed", (cfg["vocab"], W), 1.0)
    put("head", (cfg["vocab"], W))
    put("final.norm", (W, ), 0.1, 1.0)
    sd = cfg["token_side"]["dim"]
    put("side.embed", (cfg["vocab"], sd * len(cfg["layers"])), 1.0)
    for i, layer in enumerate(cfg["layers"]):
        p, mx, ml = f"l{i}.", layer["mixer"], layer.get("mlp")
        for q in "12" if ml else "1":
            put(p + f"norm{q}", (W, ), 0.2, 0.9)
            put(p + f"norm{q}b", (W, ), 0.2, 0.6)
            put(p + f"rg{q}", (W, W), 1.5 / math.sqrt(W))
            put(p + f"rg{q}.b", (W, ), 0.7, 0.3)
        put(p + "side.gate", (sd, W))
        put(p + "side.proj", (W, sd))
        put(p + "side.norm", (W, ), 0.1, 0.4)
        m = p + "mix."
        if layer["type"] == "mamba1":
            C, N, R = mx["inner"], mx["state"], mx["dt_rank"]
            put(m + "in", (2 * C, W))
            put(m + "conv", (C, mx["conv"]), 0.5)
            put(m + "conv.b", (C, ), 0.2)
            put(m + "x", (R + 2 * N, C), 1.5 / math.sqrt(C))
            put(m + "dt", (C, R), 0.7 / math.sqrt(R))
            put(m + "dt.b", (C, ), 0.7, -2.0)
            put(m + "A_log", (C, N), 0.8, -0.3)
            put(m + "D", (C, ), 0.3, 0.6)
            put(m + "o", (W, C))
        elif layer["type"] == "attention":
            H, G, d, e = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
            for n, rows in (("q", H * d), ("k", G * d), ("v", G * e), ("g", H)):
                put(m + n, (rows, W))
            put(m + "o", (W, H * e))
        else:
            H, d, r, e, R = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
            put(m + "q", (H * (d + r), W))
            put(m + "dkv", (R + r, W))
            put(m + "dkv.norm", (R, ), 0.2, 1.0)
            put(m + "uk", (H * d, R))
            put(m + "uv", (H * e, R))
            put(m + "o", (W, H * e))
        if ml and ml["kind"] == "dense":
            for n, shape in (("gate", (ml["ff"], W)), ("up", (ml["ff"], W)), ("down", (W, ml["ff"]))):
                put(p + "mlp." + n, shape)
        elif ml:
            put(p + "mlp.router", (ml["router"]["experts"], W), 1.5 / math.sqrt(W))
            for e in [f"e{j}" for j in range(ml["router"]["experts"])] + ["shared"]:
                F = (ml["shared"] if e == "shared" else ml["expert"])["ff"]
                put(p + f"mlp.{e}.up", (F, W))
                put(p + f"mlp.{e}.down", (W, F))
    if decisive:
        _decide(cfg, w, g)
    return w


def _decide(cfg, w, g):
    routed = [(f"l{i}.", la["mlp"]["router"]) for i, la in enumerate(cfg["layers"]) if (la.get("mlp") or {}).get("kind") == "moe"]
    for name in w:
        if name.endswith(("norm1b", "norm2b", "side.norm")):
            w[name][-CODE:] = 0
    for p, _ in routed:
        w[p + "mlp.router"] *= 6
        w[p + "mlp.router"][:, :-CODE] = 0
    todo = torch.arange(cfg["vocab"])
    for _ in range(2000):
        if not len(todo):
            return
        w["embed"][todo, -CODE:] = torch.randn(len(todo), CODE, generator=g).to(w["embed"].dtype)
        c = w["embed"][todo, -CODE:].double()
        near = torch.zeros(len(todo), dtype=torch.bool)
        for p, r in routed:
            count, keep, top = r["groups"]["count"], r["groups"]["keep"], r["top"]
            full = (c * w[p + "norm2"][-CODE:].double()) @ w[p + "mlp.router"][:, -CODE:].double().t()
            for shrink in (1.0, 0.6, 0.35, 0.2):   # by how much the norm may have scaled it
                z = full * shrink
                unit, n = z.std(-1) * 0.04, len(z)
                s = sigmoid(z).view(n, count, -1)
                worth = s.sort(-1, descending=True).values[..., :2].sum(-1)
                order = worth.sort(-1, descending=True).values
                if keep < count:
                    near |= order[:, keep - 1] - order[:, keep] < 0.01
                allowed = z.view(n, count, -1).masked_fill((worth < order[:, keep - 1:keep])[..., None], -math.inf).view(n, -1)
                allowed = allowed.sort(-1, descending=True).values
                if top < z.shape[1]:
                    near |= allowed[:, top - 1] - allowed[:, top] < unit
        todo = todo[near]
    raise AssertionError("no routing without near ties")


def rotation(dims, base=1000.0, factor=2.0, original=40, fast=4.0, slow=0.5):
    return {"base": base, "dims": dims, "scaling": {"factor": factor, "fast": fast, "original": original, "slow": slow}}


def mamba_layer(inner=48, state=12, dt_rank=6, conv=4, mlp=None):
    return {"type": "mamba1", "mixer": {"conv": conv, "dt_rank": dt_rank, "inner": inner, "state": state}, "mlp": mlp}


def attention_layer(heads=4, kv_heads=2, dim=16, vdim=24, size=40, rot=None, scale=None, mlp=None):
    return {"type": "attention", "mixer": {"dim": dim, "heads": heads, "kv_heads": kv_heads, "mask": {"size": size},
                                           "rot": rot or rotation(dim // 4 * 2), "scale": scale or 1.5 * dim**-0.5,
                                           "vdim": vdim}, "mlp": mlp}


def latent_layer(heads=3, dim=16, rot_dim=8, vdim=24, kv_rank=40, size=40, rot=None, scale=None, mlp=None):
    return {"type": "latent_attention", "mixer": {"dim": dim, "heads": heads, "kv_rank": kv_rank, "mask": {"size": size},
                                                  "rot": rot or rotation(rot_dim, 300.0, 3.0), "rot_dim": rot_dim,
                                                  "scale": scale or 1.5 * (dim + rot_dim)**-0.5, "vdim": vdim}, "mlp": mlp}


def dense(ff=40):
    return {"ff": ff, "kind": "dense"}


def moe(experts=6, top=2, count=3, keep=2, ff=32, shared=24, scale=1.7):
    return {"expert": {"ff": ff}, "kind": "moe", "router": {"experts": experts, "groups": {"count": count, "keep": keep},
                                                            "scale": scale, "top": top}, "shared": {"ff": shared}}


def config(layers, vocab=97, width=64, side=12, eps=1e-5):
    return {"architecture": "Nigilorn", "layers": layers, "norm": {"eps": eps}, "token_side": {"dim": side}, "vocab": vocab,
            "width": width}
