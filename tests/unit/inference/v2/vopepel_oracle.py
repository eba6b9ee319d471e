"""Plain, slow implementation of the Vopepel decoder for tests: one whole sequence at a time, one function per
mechanism, written straight from the model's equations in PyTorch on the CPU. It shares no code with the package.

Weights come as a dict of tensors under the checkpoint's names; arithmetic runs in the dtype of `cast` (float64 by
default). Nothing here is cached, paged, batched or fused."""
import math

import torch


# ------------------------------------------------------------------------------------------------ mechanisms
def layer_norm(x, w, eps):
    """Layer norm with a weight and no bias over the last dimension."""
    mean = x.mean(-1, keepdim=True)
    d = x - mean
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def head_rms_norm(x, w, eps):
    """x / rms(x) * w over the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def silu(x):
    return x / (1 + torch.exp(-x))


def causal_conv(x, taps):
    """x [n, C], taps [C, L] (last column: the current token) -> [n, C], zeros before the first token."""
    n, L = x.shape[0], taps.shape[1]
    out = torch.zeros_like(x)
    for t in range(n):
        for j in range(L):
            src = t - (L - 1 - j)
            if src >= 0:
                out[t] += taps[:, j] * x[src]
    return out


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def softplus(x):
    return torch.where(x > 30, x, torch.log1p(torch.exp(torch.clamp(x, max=30))))


def delta_rule(q, k, v, beta, g, S=None):
    """Gated delta rule, one head: q, k [n, d], v [n, e], beta, g [n] -> (o [n, e], final state [d, e])."""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=v.dtype) if S is None else S
    out = []
    for t in range(k.shape[0]):
        S = g[t] * S
        u = beta[t] * (v[t] - S.t() @ k[t])
        S = S + k[t][:, None] * u[None, :]
        out.append(S.t() @ q[t])
    return torch.stack(out), S


def softmax_attention(q, k, v, scale, softcap, chunk):
    """One head: q, k [n, d], v [n, e]. Query i sees key j <= i of its own chunk [chunk * (i // chunk), i]."""
    out = []
    for i in range(q.shape[0]):
        lo = (i // chunk) * chunk if chunk else 0
        s = (k[lo:i + 1] @ q[i]) * scale
        if softcap:
            s = softcap * torch.tanh(s / softcap)
        p = torch.exp(s - s.max())
        out.append((p / p.sum()) @ v[lo:i + 1])
    return torch.stack(out)


def clamped_glu(gate, up, limit):
    g = torch.clamp(gate, max=limit)
    u = torch.clamp(up, min=-limit, max=limit)
    return g / (1 + torch.exp(-1.702 * g)) * (u + 1)


def stream_mix(xs, y, mix, out, m):
    """xs [s, n, W] -> streams after a sublayer: x_t = sum_s mix[s, t] x_s + m out[t] y."""
    return torch.stack([sum(mix[s, t] * xs[s] for s in range(xs.shape[0])) + m * out[t] * y
                        for t in range(xs.shape[0])])


# ------------------------------------------------------------------------------------------------ layers
def delta_mixer(w, p, mx, h, eps):
    n, H, Hk, d, e = h.shape[0], mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = silu(causal_conv(h @ w[p + "q"].t(), w[p + "q.conv"])).view(n, Hk, d)
    k = silu(causal_conv(h @ w[p + "k"].t(), w[p + "k.conv"])).view(n, Hk, d)
    v = silu(causal_conv(h @ w[p + "v"].t(), w[p + "v.conv"])).view(n, H, e)
    q, k = unit(q) * d**-0.5, unit(k)
    beta = 1 / (1 + torch.exp(-(h @ w[p + "b"].t())))
    g = torch.exp(-torch.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].t() + w[p + "dt_bias"]))
    gate = silu(h @ w[p + "g"].t()).view(n, H, e)
    rep = H // Hk
    o = torch.stack([delta_rule(q[:, i // rep], k[:, i // rep], v[:, i], beta[:, i], g[:, i])[0]
                     for i in range(H)], 1)
    o = head_rms_norm(o, w[p + "norm"], eps) * gate
    return o.reshape(n, H * e) @ w[p + "o"].t()


def attention_mixer(w, p, mx, h, eps, v_first):
    """Returns (output, v_first after this layer)."""
    n, H, G, d, e = h.shape[0], mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = head_rms_norm((h @ w[p + "q"].t()).view(n, H, d), w[p + "q.norm"], eps)
    k = head_rms_norm((h @ w[p + "k"].t()).view(n, G, d), w[p + "k.norm"], eps)
    v = (h @ w[p + "v"].t()).view(n, G, e)
    if mx.get("v_mix"):
        if v_first is None:
            v_first = v
        else:
            lam = w[p + "vmix"].reshape(())
            v = (1 - lam) * v + lam * v_first
    rep = H // G
    chunk = (mx.get("mask") or {}).get("size", 0)
    o = torch.stack([softmax_attention(q[:, i], k[:, i // rep], v[:, i // rep], mx["scale"], mx.get("softcap"),
                                       chunk) for i in range(H)], 1)
    return o.reshape(n, H * e) @ w[p + "o"].t(), v_first


def dense_mlp(w, p, ml, h):
    return clamped_glu(h @ w[p + "gate"].t(), h @ w[p + "up"].t(), ml["limit"]) @ w[p + "down"].t()


def forward(cfg, weights, tokens, cast=torch.float64, trace=None):
    """Logits [n, vocab] of one sequence; `trace` (a list) receives the sum of the streams after every layer."""
    w = {k: v.to(cast) for k, v in weights.items()}
    eps, m, s = cfg["norm"]["eps"], cfg["residual_mult"], cfg["streams"]
    xs = w["embed"][torch.as_tensor(tokens)][None].repeat(s, 1, 1)
    v_first = None
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        for q, kind in ((1, layer["type"]), (2, layer.get("mlp"))):
            if kind is None:
                continue
            u = sum(w[f"{p}hc{q}.in"][j] * xs[j] for j in range(s))
            h = layer_norm(u, w[f"{p}norm{q}"], eps)
            if q == 2:
                y = dense_mlp(w, p + "mlp.", layer["mlp"], h)
            elif kind == "delta":
                y = delta_mixer(w, p + "mix.", layer["mixer"], h, eps)
            else:
                y, v_first = attention_mixer(w, p + "mix.", layer["mixer"], h, eps, v_first)
            xs = stream_mix(xs, y, w[f"{p}hc{q}.mix"], w[f"{p}hc{q}.out"], m)
        if trace is not None:
            trace.append(xs.sum(0))
    return layer_norm(xs.sum(0), w["final.norm"], eps) @ w["head"].t()


# ------------------------------------------------------------------------------------------------ test models
def random_model(cfg, seed=0, dtype=torch.bfloat16, peak=1.0):
    """Random weights for a config. `peak` scales the q / k norm weights of the attention layers (a larger value makes
    single keys stand out among many)."""
    g = torch.Generator().manual_seed(seed)
    W, w = cfg["width"], {}

    def put(name, shape, std=None, mean=0.0):
        std = std if std is not None else 1 / math.sqrt(shape[-1])
        w[name] = (torch.randn(shape, generator=g) * std + mean).to(dtype)

    put("embed", (cfg["vocab"], W), 1.0)
    put("head", (cfg["vocab"], W))
    put("final.norm", (W, ), 0.1, 1.0)
    s = cfg["streams"]
    for i, layer in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", layer["mixer"]
        H, Hk, d, e = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
        for q in (1, 2) if layer.get("mlp") else (1, ):
            put(f"{p}norm{q}", (W, ), 0.2, 1.0)
            put(f"{p}hc{q}.in", (s, ), 0.3, 0.5)
            put(f"{p}hc{q}.out", (s, ), 0.3, 0.7)
            w[f"{p}hc{q}.mix"] = (torch.eye(s) * 0.8 + torch.randn(s, s, generator=g) * 0.15).to(dtype)
        p += "mix."
        if layer["type"] == "delta":
            for n, c in (("q", Hk * d), ("k", Hk * d), ("v", H * e)):
                put(p + n, (c, W))
                put(p + n + ".conv", (c, mx["conv"]), 0.5)
            put(p + "b", (H, W))
            put(p + "a", (H, W))
            put(p + "g", (H * e, W))
            put(p + "A_log", (H, ), 0.7, -1.0)
            put(p + "dt_bias", (H, ), 0.5, -2.0)
            put(p + "norm", (e, ), 0.2, 1.0)
        else:
            put(p + "q", (H * d, W))
            put(p + "k", (Hk * d, W))
            put(p + "v", (Hk * e, W))
            put(p + "q.norm", (d, ), 0.2, peak)
            put(p + "k.norm", (d, ), 0.2, peak)
            if mx.get("v_mix"):
                w[p + "vmix"] = torch.tensor(0.3 + 0.1 * (i % 3)).to(dtype)
        put(p + "o", (W, H * e))
        if layer.get("mlp"):
            p, F = f"l{i}.mlp.", layer["mlp"]["ff"]
            put(p + "gate", (F, W))
            put(p + "up", (F, W))
            put(p + "down", (W, F))
    return w


def delta_layer(heads=4, kv_heads=2, dim=16, vdim=24, conv=4, ff=72, limit=0.9):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv},
            "mlp": {"kind": "dense", "ff": ff, "limit": limit} if ff else None}


def attention_layer(heads=4, kv_heads=2, dim=32, vdim=16, size=24, scale=0.2, softcap=9.0, v_mix=True, ff=72,
                    limit=0.9):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": size},
                      "scale": scale, "softcap": softcap, "v_mix": v_mix},
            "mlp": {"kind": "dense", "ff": ff, "limit": limit} if ff else None}


def config(layers, vocab=97, width=64, streams=3, residual_mult=0.6, eps=1e-5):
    return {"architecture": "Vopepel", "layers": layers, "norm": {"eps": eps}, "residual_mult": residual_mult,
            "streams": streams, "vocab": vocab, "width": width}
