"""Plain, slow implementation of the Lefisun decoder for tests: one whole sequence at a time, one function per mechanism,
written straight from the model's equations in PyTorch on the CPU. It shares no code with the package.

Weights come as a dict of tensors under the checkpoint's names; arithmetic runs in the dtype of `cast` (float64 by
default). Nothing here is cached, paged, batched, chunked or fused. Under `Rounded()` the operands and results of the
projections are rounded to bf16: what a model in 16 bits cannot do better than."""
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


def log_sigmoid(x):
    """-log(1 + e^-x), without overflow on either side."""
    return torch.minimum(x, torch.zeros_like(x)) - torch.log1p(torch.exp(-x.abs()))


def soft_cap(x, cap):
    return cap * torch.tanh(x / cap)


def rotate(x, dims, base, factor=1.0, first=0):
    """x [n, d]: row i sits at position first + i; pairs (j, j + dims / 2) of the first `dims` elements turn by
    position * base^(-2 j / dims) / factor."""
    half = dims // 2
    out = x.clone()
    for i in range(x.shape[0]):
        for j in range(half):
            a = (first + i) * base**(-2 * j / dims) / factor
            u, v = x[i, j], x[i, j + half]
            out[i, j] = u * math.cos(a) - v * math.sin(a)
            out[i, j + half] = v * math.cos(a) + u * math.sin(a)
    return out


def chunked_attention(q, k, v, scale, chunk):
    """One head: q, k [n, d], v [n, e]. Query i sees the keys j <= i of its own chunk; the weights share their sum with a
    score of zero that carries no value."""
    out = []
    for i in range(q.shape[0]):
        lo = i // chunk * chunk if chunk else 0
        s = (k[lo:i + 1] @ q[i]) * scale
        m = torch.clamp(s.max(), min=0)
        p = torch.exp(s - m)
        out.append((p / (torch.exp(-m) + p.sum())) @ v[lo:i + 1])
    return torch.stack(out)


def matrix_memory(q, k, v, log_in, log_forget):
    """One head: q, k [n, d], v [n, e], log gates [n] -> [n, e]. State and normaliser are kept relative to e^m."""
    S, z, m = torch.zeros(k.shape[1], v.shape[1], dtype=v.dtype), torch.zeros(k.shape[1], dtype=v.dtype), torch.zeros((), dtype=v.dtype)
    out = []
    for t in range(k.shape[0]):
        m_new = torch.maximum(log_forget[t] + m, log_in[t])
        keep, add = torch.exp(log_forget[t] + m - m_new), torch.exp(log_in[t] - m_new)
        S, z, m = keep * S + add * k[t][:, None] * v[t][None, :], keep * z + add * k[t], m_new
        out.append((S.t() @ q[t]) / (torch.maximum((z @ q[t]).abs(), torch.exp(-m)) + 1e-6))
    return torch.stack(out)


def decayed_scan(q, k, v, decay):
    """One head: S_t = decay S_(t-1) + k_t v_t^T, o_t = S_t^T q_t."""
    S, out = torch.zeros(k.shape[1], v.shape[1], dtype=v.dtype), []
    for t in range(k.shape[0]):
        S = decay * S + k[t][:, None] * v[t][None, :]
        out.append(S.t() @ q[t])
    return torch.stack(out)


def route(z, top, groups, keep):
    """Router logits z [n, E] -> (experts [n, top], weights [n, top]): the best experts of the `keep` best groups (a group is
    as good as its best member), weighted by their softmax over all experts."""
    s = torch.softmax(z, -1)
    n, E = s.shape
    best = s.view(n, groups, E // groups).max(-1).values
    allowed = torch.zeros(n, groups, dtype=torch.bool).scatter_(1, best.topk(keep, -1).indices, True)
    e = s.masked_fill(~allowed.repeat_interleave(E // groups, 1), -1.0).topk(top, -1).indices
    w = s.gather(1, e)
    return e, w / (w.sum(-1, keepdim=True) + 1e-20)


# ------------------------------------------------------------------------------------------------ layers
def attention_side(w, p, mx, h, eps):
    n, H, G, d, e = h.shape[0], mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q, k, v = (project(h, w[p + c]) + w[p + c + ".b"] for c in "qkv")
    q, k = rms(q, eps) * w[p + "q.norm"], rms(k, eps) * w[p + "k.norm"]
    q, k, v = q.view(n, H, d), k.view(n, G, d), v.view(n, G, e)
    rot = mx["rot"]
    turn = lambda x: rotate(x, rot["dims"], rot["base"], rot["scaling"]["factor"])
    ks = [turn(k[:, g]) for g in range(G)]
    out = [chunked_attention(turn(q[:, i]), ks[i // (H // G)], v[:, i // (H // G)], mx["scale"], mx["mask"]["size"])
           for i in range(H)]
    return torch.stack(out, 1).reshape(n, H * e)


def memory_side(w, p, mx, h, eps):
    n, H, d, e, cap = h.shape[0], mx["heads"], mx["dim"], mx["vdim"], mx["gate_cap"]
    q, k = project(h, w[p + "q"]).view(n, H, d) * d**-0.5, project(h, w[p + "k"]).view(n, H, d)
    v = project(h, w[p + "v"]).view(n, H, e)
    i = soft_cap(project(h, w[p + "i"]) + w[p + "i.b"], cap)
    f = log_sigmoid(soft_cap(project(h, w[p + "f"]) + w[p + "f.b"], cap))
    o = torch.stack([matrix_memory(q[:, j], k[:, j], v[:, j], i[:, j], f[:, j]) for j in range(H)], 1)
    return rms(o, eps).reshape(n, H * e) * w[p + "norm"] * sigmoid(project(h, w[p + "g"]))


def parallel_mixer(w, p, mx, h, eps):
    """Both sides read the same input. (Under `Rounded()` each is rounded on its way into its output projection.)"""
    left = project(attention_side(w, p + "left.", mx["left"], h, eps), w[p + "left.o"])
    right = project(memory_side(w, p + "right.", mx["right"], h, eps), w[p + "right.o"])
    return mx["left_scale"] * left + mx["right_scale"] * right


def retention_mixer(w, p, mx, h, eps):
    n, H, d, e, rot = h.shape[0], mx["heads"], mx["dim"], mx["vdim"], mx["rot"]
    q, k = (project(h, w[p + c]).view(n, H, d) for c in "qk")
    v = project(h, w[p + "v"]).view(n, H, e)
    turn = lambda x: rotate(x, rot["dims"], rot["base"])
    o = torch.stack([decayed_scan(turn(q[:, i]), turn(k[:, i]) * d**-0.5, v[:, i], mx["decay"][i]) for i in range(H)], 1)
    return project(rms(o, eps).reshape(n, H * e) * silu(project(h, w[p + "g"])), w[p + "o"])


MIXERS = {"parallel": parallel_mixer, "retention": retention_mixer}


def experts(w, p, ml, h):
    r = ml["router"]
    e, wt = route(h @ w[p + "router"].t(), r["top"], r["groups"]["count"], r["groups"]["keep"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for j in range(r["top"]):
            q, x = f"{p}e{int(e[t, j])}.", h[t:t + 1]
            y = project(silu(project(x, w[q + "gate"])) * project(x, w[q + "up"]), w[q + "down"])
            out[t] += wt[t, j] * y[0]
    return out


def forward(cfg, weights, tokens, cast=torch.float64, trace=None):
    """Logits [n, vocab] of one sequence; `trace` (a list) receives the residual after every layer."""
    w = {k: v.to(cast) for k, v in weights.items()}
    eps, ids = cfg["norm"]["eps"], torch.as_tensor(tokens).long()
    x = w["embed"][ids] * cfg["embedding"]["scale"]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + MIXERS[layer["type"]](w, p + "mix.", layer["mixer"], rms(x, eps) * w[p + "norm1"], eps)
        if layer.get("mlp"):
            x = x + experts(w, p + "mlp.", layer["mlp"], rms(x, eps) * w[p + "norm2"])
        if trace is not None:
            trace.append(x)
    return project(rms(x, eps) * w["final.norm"], w["embed"])


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

    put("embed", (cfg["vocab"], W), 1.0 / cfg["embedding"]["scale"])
    put("final.norm", (W, ), 0.1, 1.0 / math.sqrt(W))
    w["final.norm"] *= cfg["embedding"]["scale"]
    for i, layer in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", layer["mixer"]
        put(p + "norm1", (W, ), 0.2, 0.9)
        if layer["type"] == "parallel":
            le, ri = mx["left"], mx["right"]
            q = p + "mix.left."
            for n, rows in (("q", le["heads"] * le["dim"]), ("k", le["kv_heads"] * le["dim"]), ("v", le["kv_heads"] * le["vdim"])):
                put(q + n, (rows, W))
                put(q + n + ".b", (rows, ), 0.5)
            put(q + "q.norm", (le["heads"] * le["dim"], ), 0.2, 1.0)
            put(q + "k.norm", (le["kv_heads"] * le["dim"], ), 0.2, 1.0)
            put(q + "o", (W, le["heads"] * le["vdim"]))
            q, H = p + "mix.right.", ri["heads"]
            for n, rows in (("q", H * ri["dim"]), ("k", H * ri["dim"]), ("v", H * ri["vdim"]), ("g", H * ri["vdim"]), ("i", H),
                            ("f", H)):
                put(q + n, (rows, W))
            put(q + "i.b", (H, ), 1.0)
            put(q + "f.b", (H, ), 1.5, 2.0)
            put(q + "norm", (H * ri["vdim"], ), 0.2, 1.0)
            put(q + "o", (W, H * ri["vdim"]))
        else:
            H = mx["heads"]
            for n, rows in (("q", H * mx["dim"]), ("k", H * mx["dim"]), ("v", H * mx["vdim"]), ("g", H * mx["vdim"])):
                put(p + f"mix.{n}", (rows, W))
            put(p + "mix.o", (W, H * mx["vdim"]))
        if layer.get("mlp"):
            F, E = layer["mlp"]["expert"]["ff"], layer["mlp"]["router"]["experts"]
            put(p + "norm2", (W, ), 0.2, 0.9)
            put(p + "mlp.router", (E, W), 1.5 / math.sqrt(W))
            for e in range(E):
                put(p + f"mlp.e{e}.gate", (F, W))
                put(p + f"mlp.e{e}.up", (F, W))
                put(p + f"mlp.e{e}.down", (W, F))
    if decisive:
        _decide(cfg, w, g)
    return w


def _decide(cfg, w, g):
    routed = [(f"l{i}.", la["mlp"]["router"]) for i, la in enumerate(cfg["layers"]) if la.get("mlp")]
    for name in w:
        if name.endswith(("mix.o", "left.o", "right.o", ".down")):
            w[name][-CODE:] = 0
    for p, _ in routed:
        w[p + "mlp.router"] *= 6
        w[p + "mlp.router"][:, :-CODE] = 0
    todo = torch.arange(cfg["vocab"])
    for _ in range(500):
        w["embed"][todo, -CODE:] = (torch.randn(len(todo), CODE, generator=g) / cfg["embedding"]["scale"]).to(w["embed"].dtype)
        c = w["embed"][todo, -CODE:].double()
        near = torch.zeros(len(todo), dtype=torch.bool)
        for p, r in routed:
            z = (c * w[p + "norm2"][-CODE:].double()) @ w[p + "mlp.router"][:, -CODE:].double().t()
            unit = z.std(-1) * 0.05
            n, (count, keep, top) = len(todo), (r["groups"]["count"], r["groups"]["keep"], r["top"])
            best = z.view(n, count, -1).max(-1).values.sort(-1, descending=True).values
            if keep < count:
                near |= best[:, keep - 1] - best[:, keep] < unit
            allowed = z.view(n, count, -1).masked_fill((z.view(n, count, -1).max(-1).values < best[:, keep - 1:keep])[..., None],
                                                       -math.inf).view(n, -1).sort(-1, descending=True).values
            if top < z.shape[1]:
                near |= allowed[:, top - 1] - allowed[:, top] < unit
        todo = todo[near]
        if not len(todo):
            return
    raise AssertionError("no routing without near ties")


def parallel_layer(heads=4, kv_heads=2, dim=16, vdim=24, size=40, rot=8, base=1000.0, factor=2.0, scale=None, left_scale=0.7,
                   right_scale=0.6, r_heads=2, r_dim=16, r_vdim=24, cap=8.0, mlp=None):
    return {"type": "parallel",
            "mixer": {"left": {"dim": dim, "heads": heads, "kv_heads": kv_heads, "mask": {"size": size},
                               "rot": {"base": base, "dims": rot, "scaling": {"factor": factor}},
                               "scale": scale or dim**-0.5, "vdim": vdim},
                      "left_scale": left_scale, "right": {"dim": r_dim, "gate_cap": cap, "heads": r_heads, "vdim": r_vdim},
                      "right_scale": right_scale}, "mlp": mlp}


def retention_layer(heads=3, dim=16, vdim=24, decay=None, rot=None, base=5000.0, mlp=None):
    decay = decay or [1 - 2.0**-(2 * i + 3) for i in range(heads)]
    return {"type": "retention", "mixer": {"decay": decay, "dim": dim, "heads": heads,
                                           "rot": {"base": base, "dims": dim if rot is None else rot}, "vdim": vdim}, "mlp": mlp}


def moe(experts=6, top=2, count=3, keep=2, ff=32):
    return {"expert": {"ff": ff}, "kind": "moe", "router": {"experts": experts, "groups": {"count": count, "keep": keep},
                                                            "top": top}}


def config(layers, vocab=97, width=64, scale=1.7, eps=1e-5):
    return {"architecture": "Lefisun", "embedding": {"scale": scale}, "layers": layers, "norm": {"eps": eps}, "vocab": vocab,
            "width": width}
