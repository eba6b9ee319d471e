"""Plain, slow implementation of the Perelorn decoder for tests: one whole sequence at a time, one function per
mechanism, written straight from the model's equations in PyTorch on the CPU. It shares no code with the package.

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
def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def silu(x):
    return x / (1 + torch.exp(-x))


def sigmoid(x):
    return 1 / (1 + torch.exp(-x))


def softplus(x):
    return torch.where(x > 30, x, torch.log1p(torch.exp(torch.clamp(x, max=30))))


def gelu_erf(x):
    return 0.5 * x * (1 + torch.erf(x / math.sqrt(2)))


def gelu_tanh(x):
    return 0.5 * x * (1 + torch.tanh(math.sqrt(2 / math.pi) * (x + 0.044715 * x**3)))


def causal_conv(x, taps, bias):
    """x [n, C], taps [C, L] (last column: the current token), bias [C] -> [n, C], zeros before the first token."""
    n, L = x.shape[0], taps.shape[1]
    out = bias.expand(n, -1).clone()
    for t in range(n):
        for j in range(L):
            src = t - (L - 1 - j)
            if src >= 0:
                out[t] += taps[:, j] * x[src]
    return out


def rotate(x, dims, base, first=0):
    """x [n, d]: row i sits at position first + i; pairs (j, j + dims / 2) of the first `dims` elements turn by
    position * base^(-2 j / dims)."""
    half = dims // 2
    out = x.clone()
    for i in range(x.shape[0]):
        for j in range(half):
            a = (first + i) * base**(-2 * j / dims)
            u, v = x[i, j], x[i, j + half]
            out[i, j] = u * math.cos(a) - v * math.sin(a)
            out[i, j + half] = v * math.cos(a) + u * math.sin(a)
    return out


def sink_attention(q, k, v, scale, sink):
    """One head: q, k [n, d], v [n, e]. Query i sees every key j <= i; the weights share their sum with exp(sink)."""
    out = []
    for i in range(q.shape[0]):
        s = (k[:i + 1] @ q[i]) * scale
        m = torch.maximum(s.max(), sink)
        p = torch.exp(s - m)
        out.append((p / (p.sum() + torch.exp(sink - m))) @ v[:i + 1])
    return torch.stack(out)


def decayed_scan(q, k, v, decay, step, S=None):
    """One head: S_t = decay_t S_(t-1) + step_t k_t v_t^T, o_t = S_t^T q_t. q, k [n, d], v [n, e], decay / step [n]
    -> (o [n, e], final state [d, e])."""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=v.dtype) if S is None else S
    out = []
    for t in range(k.shape[0]):
        S = decay[t] * S + step[t] * k[t][:, None] * v[t][None, :]
        out.append(S.t() @ q[t])
    return torch.stack(out), S


def grouped_rms(x, parts, eps):
    """x [n, C]: every one of the `parts` equal parts of a row by its own root mean square."""
    y = x.view(x.shape[0], parts, -1)
    return (y / torch.sqrt((y * y).mean(-1, keepdim=True) + eps)).reshape(x.shape)


# ------------------------------------------------------------------------------------------------ layers
def mamba2_mixer(w, p, mx, h, eps):
    n, H, e, N, G = h.shape[0], mx["heads"], mx["vdim"], mx["state"], mx["groups"]
    inner = H * e
    z, x, B, C, dt = torch.split(project(h, w[p + "in"]), [inner, inner, G * N, G * N, H], -1)
    xbc = silu(causal_conv(torch.cat([x, B, C], -1), w[p + "conv"], w[p + "conv.b"]))
    x, B, C = torch.split(xbc, [inner, G * N, G * N], -1)
    x, B, C = x.view(n, H, e), B.view(n, G, N), C.view(n, G, N)
    dt = softplus(dt + w[p + "dt_bias"])
    decay = torch.exp(-torch.exp(w[p + "A_log"]) * dt)
    y = []
    for i in range(H):
        g = i // (H // G)
        o, _ = decayed_scan(C[:, g], B[:, g], x[:, i], decay[:, i], dt[:, i])
        y.append(o + w[p + "D"][i] * x[:, i])
    y = torch.stack(y, 1).reshape(n, inner) * silu(z)
    return project(grouped_rms(y, mx["norm_groups"], eps) * w[p + "norm"], w[p + "o"])


def lightning_mixer(w, p, mx, h, eps):
    n, H, d, e = h.shape[0], mx["heads"], mx["dim"], mx["vdim"]
    q = silu(project(h, w[p + "q"])).view(n, H, d)
    k = silu(project(h, w[p + "k"])).view(n, H, d)
    v = silu(project(h, w[p + "v"])).view(n, H, e)
    one = torch.ones(n, dtype=h.dtype)
    o = torch.stack([decayed_scan(q[:, i], k[:, i], v[:, i], mx["decay"][i] * one, one)[0] for i in range(H)], 1)
    o = rms_norm(o.reshape(n, H * e), w[p + "norm"], eps) * sigmoid(project(h, w[p + "g"]))
    return project(o, w[p + "o"])


def latent_mixer(w, p, mx, h, eps):
    n, H, d, r, e, R = h.shape[0], mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
    q = project(rms_norm(project(h, w[p + "dq"]), w[p + "dq.norm"], eps), w[p + "uq"]).view(n, H, d + r)
    down = project(h, w[p + "dkv"])
    c = rms_norm(down[:, :R], w[p + "dkv.norm"], eps)
    kr = rotate(down[:, R:], mx["rot"]["dims"], mx["rot"]["base"])
    k, v = project(c, w[p + "uk"]).view(n, H, d), project(c, w[p + "uv"]).view(n, H, e)
    out = []
    for i in range(H):
        qr = rotate(q[:, i, d:], mx["rot"]["dims"], mx["rot"]["base"])
        out.append(sink_attention(torch.cat([q[:, i, :d], qr], -1), torch.cat([k[:, i], kr], -1), v[:, i], mx["scale"],
                                  w[p + "sink"][i]))
    return project(torch.stack(out, 1).reshape(n, H * e), w[p + "o"])


MIXERS = {"mamba2": mamba2_mixer, "lightning": lightning_mixer, "latent_attention": latent_mixer}


def token_side(w, p, dim, i, x, tokens, eps):
    """The layer's own embedding of each token, gated by the residual and added to it."""
    e = w["side.embed"][tokens][:, i * dim:(i + 1) * dim]
    g = gelu_tanh(project(x, w[p + "side.gate"])) * e
    return rms_norm(project(g, w[p + "side.proj"]), w[p + "side.norm"], eps)


def forward(cfg, weights, tokens, cast=torch.float64, trace=None):
    """Logits [n, vocab] of one sequence; `trace` (a list) receives the residual after every layer."""
    w = {k: v.to(cast) for k, v in weights.items()}
    eps, ids = cfg["norm"]["eps"], torch.as_tensor(tokens).long()
    x = w["embed"][ids]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + rms_norm(MIXERS[layer["type"]](w, p + "mix.", layer["mixer"], x, eps), w[p + "norm1"], eps)
        if layer.get("mlp"):
            y = project(gelu_erf(project(x, w[p + "mlp.up"])), w[p + "mlp.down"])
            x = x + rms_norm(y, w[p + "norm2"], eps)
        x = x + token_side(w, p, cfg["token_side"]["dim"], i, x, ids, eps)
        if trace is not None:
            trace.append(x)
    return project(rms_norm(x, w["final.norm"], eps), w["head"]) * cfg["logit_scale"]


# ------------------------------------------------------------------------------------------------ test models
def random_model(cfg, seed=0, dtype=torch.bfloat16, peak=1.0):
    """Random weights for a config. `peak` scales the latent attention's query projection (a larger value makes single
    keys stand out among many)."""
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
        p, mx = f"l{i}.", layer["mixer"]
        put(p + "norm1", (W, ), 0.2, 0.8)
        put(p + "side.gate", (sd, W))
        put(p + "side.proj", (W, sd))
        put(p + "side.norm", (W, ), 0.1, 0.4)
        if layer.get("mlp"):
            put(p + "norm2", (W, ), 0.2, 0.6)
            put(p + "mlp.up", (layer["mlp"]["ff"], W))
            put(p + "mlp.down", (W, layer["mlp"]["ff"]))
        p += "mix."
        H, e = mx["heads"], mx["vdim"]
        put(p + "o", (W, H * e))
        if layer["type"] == "mamba2":
            ch = H * e + 2 * mx["groups"] * mx["state"]
            put(p + "in", (H * e + ch + H, W))
            put(p + "conv", (ch, mx["conv"]), 0.5)
            put(p + "conv.b", (ch, ), 0.2)
            put(p + "dt_bias", (H, ), 0.7, -2.0)
            put(p + "A_log", (H, ), 0.8, -0.5)
            put(p + "D", (H, ), 0.3, 0.6)
            put(p + "norm", (H * e, ), 0.2, 1.0)
        elif layer["type"] == "lightning":
            put(p + "q", (H * mx["dim"], W))
            put(p + "k", (H * mx["dim"], W))
            put(p + "v", (H * e, W))
            put(p + "g", (H * e, W))
            put(p + "norm", (H * e, ), 0.2, 1.0)
        else:
            d, r, R, Q = mx["dim"], mx["rot_dim"], mx["kv_rank"], mx["q_rank"]
            put(p + "dq", (Q, W))
            put(p + "dq.norm", (Q, ), 0.2, 1.0)
            put(p + "uq", (H * (d + r), Q), peak / math.sqrt(Q))
            put(p + "dkv", (R + r, W))
            put(p + "dkv.norm", (R, ), 0.2, 1.0)
            put(p + "uk", (H * d, R))
            put(p + "uv", (H * e, R))
            put(p + "sink", (H, ), 0.8, 0.5)
    return w


def mamba2_layer(heads=4, groups=2, state=16, vdim=24, conv=4, norm_groups=2, ff=0):
    return {"type": "mamba2", "mixer": {"conv": conv, "groups": groups, "heads": heads, "norm_groups": norm_groups,
                                        "state": state, "vdim": vdim}, "mlp": {"ff": ff, "kind": "dense"} if ff else None}


def lightning_layer(heads=3, dim=16, vdim=24, decay=None, ff=0):
    decay = decay or [math.exp(-2.0**-(2 * i + 1)) for i in range(heads)]
    return {"type": "lightning", "mixer": {"decay": decay, "dim": dim, "heads": heads, "vdim": vdim},
            "mlp": {"ff": ff, "kind": "dense"} if ff else None}


def latent_layer(heads=3, dim=16, rot_dim=8, vdim=24, kv_rank=40, q_rank=32, base=1000.0, scale=None, ff=56):
    return {"type": "latent_attention",
            "mixer": {"dim": dim, "heads": heads, "kv_rank": kv_rank, "q_rank": q_rank, "rot": {"base": base,
                                                                                              "dims": rot_dim},
                      "rot_dim": rot_dim, "scale": scale or (dim + rot_dim)**-0.5, "vdim": vdim},
            "mlp": {"ff": ff, "kind": "dense"} if ff else None}


def config(layers, vocab=97, width=64, side=12, logit_scale=1.5, eps=1e-5):
    return {"architecture": "Perelorn", "layers": layers, "logit_scale": logit_scale, "norm": {"eps": eps},
            "token_side": {"dim": side}, "vocab": vocab, "width": width}
