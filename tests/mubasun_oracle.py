"""Plain, slow Mubasun forward pass: the oracle of the Mubasun tests.

One function per mechanism, straight from the equations, whole sequences at a
time, no cache, no batching, no kernels. It shares no code with bloombee_amd
(only torch) and computes in the dtype of the weights it is given; the tests
pass float64 or float32.

`w` is a dict {tensor name: tensor}, `cfg` the model's configuration dict.
"""
import math

import torch


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def grouped_rms(x, weight, groups, eps):
    """Every one of `groups` consecutive parts by its own root mean square."""
    parts = x.reshape(*x.shape[:-1], groups, x.shape[-1] // groups)
    return rms(parts, eps).reshape(x.shape) * weight


def slopes(heads, dtype):
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)],
                        dtype=dtype)


def xielu(z, p, q):
    softplus = lambda t: math.log1p(math.exp(-abs(t))) + max(t, 0.0)
    pos = softplus(float(p)) * z * z + 0.5 * z
    neg = (0.5 + softplus(float(q))) * (torch.expm1(z.clamp(max=0)) - z) + 0.5 * z
    return torch.where(z > 0, pos, neg)


def silu(z):
    return z / (1 + torch.exp(-z))


def keys_values(h, w, pre, mx, eps):
    """Keys (normed over the whole projection) and values, [T, G, dim]."""
    T, G = h.shape[0], mx["kv_heads"]
    k = rms(h @ w[pre + "k"].T, eps) * w[pre + "k.norm"]
    v = h @ w[pre + "v"].T
    return k.reshape(T, G, mx["dim"]), v.reshape(T, G, mx["vdim"])


def visible(T, size):
    """[T, T] bool: query i (row) sees key j (column)."""
    d = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    return (d >= 0) & (d < size) if size else d >= 0


def attend(q, k, v, scale, size):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] -> [T, H, vdim]."""
    T, H, _ = q.shape
    G = k.shape[1]
    sl = slopes(H, q.dtype)
    dist = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).to(q.dtype)
    see = visible(T, size)
    out = torch.empty(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale - sl[h] * dist
        out[:, h] = torch.softmax(s.masked_fill(~see, -math.inf), -1) @ v[:, g]
    return out


def mixer(h, w, pre, mx, eps, kv):
    """The attention sublayer's output for normed input h [T, width]."""
    T, H = h.shape[0], mx["heads"]
    q = (rms(h @ w[pre + "q"].T, eps) * w[pre + "q.norm"]).reshape(T, H, mx["dim"])
    size = (mx.get("mask") or {}).get("size")
    o = attend(q, kv[0], kv[1], mx["scale"], size).reshape(T, -1)
    return (o * torch.sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T


def dense_mlp(h, w, pre):
    p, q = w[pre + "act"]
    return xielu(h @ w[pre + "up"].T, p, q) @ w[pre + "down"].T


def glu(h, w, pre):
    return (silu(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def route(h, w, pre, rt):
    """[T, experts + identity] weights, zero for the ones not chosen."""
    s = torch.softmax(h @ w[pre + "router"].T, -1)
    choice = s + w[pre + "correction"]
    chosen = torch.zeros_like(s, dtype=torch.bool)
    for t in range(h.shape[0]):
        chosen[t, torch.topk(choice[t], rt["top"]).indices] = True
    return torch.where(chosen, s * rt["scale"], torch.zeros_like(s))


def moe(h, w, pre, mlp):
    rt = mlp["router"]
    wt = route(h, w, pre, rt)
    E = rt["experts"]
    out = torch.zeros_like(h)
    for e in range(E):
        rows = (wt[:, e] != 0).nonzero(as_tuple=True)[0]
        if len(rows):
            out[rows] += wt[rows, e:e + 1] * glu(h[rows], w, f"{pre}e{e}.")
    out += wt[:, E:].sum(-1, keepdim=True) * h          # identity experts
    if mlp.get("shared"):
        out += torch.sigmoid(h @ w[pre + "shared.sg"].T) * glu(h, w, pre + "shared.")
    return out


def forward(tokens, w, cfg, collect=None):
    """Logits [T, vocab] of one sequence; collect gets x after every layer."""
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    x = w["embed"][tokens] + w["pos"][: len(tokens)]
    kvs = []
    for i, layer in enumerate(cfg["layers"]):
        mx, mlp = layer["mixer"], layer["mlp"]
        h = grouped_rms(x, w[f"l{i}.norm1"], groups, eps)
        src = mx.get("kv_from")
        kvs.append(kvs[src] if src is not None
                   else keys_values(h, w, f"l{i}.mix.", mx, eps))
        y = mixer(h, w, f"l{i}.mix.", mx, eps, kvs[i])
        if mlp is not None:
            y = y + (dense_mlp(h, w, f"l{i}.mlp.") if mlp["kind"] == "dense"
                     else moe(h, w, f"l{i}.mlp.", mlp))
        x = x + y
        if collect is not None:
            collect.append(x)
    return grouped_rms(x, w["final.norm"], groups, eps) @ w["head"].T


# ---------------------------------------------------------------------------
# small random models
# ---------------------------------------------------------------------------

def tensor_shapes(cfg):
    D = cfg["width"]
    s = {"embed": (cfg["vocab"], D), "pos": (cfg["max_positions"], D),
         "final.norm": (D,), "head": (cfg["vocab"], D)}
    for i, layer in enumerate(cfg["layers"]):
        mx, mlp = layer["mixer"], layer["mlp"]
        p = f"l{i}."
        s[p + "norm1"] = (D,)
        s[p + "mix.q"] = (mx["heads"] * mx["dim"], D)
        s[p + "mix.q.norm"] = (mx["heads"] * mx["dim"],)
        s[p + "mix.g"] = (mx["heads"] * mx["vdim"], D)
        s[p + "mix.o"] = (D, mx["heads"] * mx["vdim"])
        if mx.get("kv_from") is None:
            s[p + "mix.k"] = (mx["kv_heads"] * mx["dim"], D)
            s[p + "mix.k.norm"] = (mx["kv_heads"] * mx["dim"],)
            s[p + "mix.v"] = (mx["kv_heads"] * mx["vdim"], D)
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            s[p + "mlp.up"] = (mlp["ff"], D)
            s[p + "mlp.down"] = (D, mlp["ff"])
            s[p + "mlp.act"] = (2,)
            continue
        rt = mlp["router"]
        for e in range(rt["experts"]):
            s[p + f"mlp.e{e}.gate"] = s[p + f"mlp.e{e}.up"] = (mlp["expert"]["ff"], D)
            s[p + f"mlp.e{e}.down"] = (D, mlp["expert"]["ff"])
        n = rt["experts"] + rt["identity"]
        s[p + "mlp.router"] = (n, D)
        s[p + "mlp.correction"] = (n,)
        if mlp.get("shared"):
            s[p + "mlp.shared.gate"] = s[p + "mlp.shared.up"] = (mlp["shared"]["ff"], D)
            s[p + "mlp.shared.down"] = (D, mlp["shared"]["ff"])
            s[p + "mlp.shared.sg"] = (1, D)
    return s


def random_weights(cfg, seed=0):
    """bf16-representable float32 weights of a lively scale.

    Routing must not hang on a rounding, or a 16-bit run would rightly differ
    from the oracle. So the last norm group (the last sixth, if there is one
    group) carries a code of +-1 per token: nothing writes to it after the
    embedding, and the routers read nothing else."""
    gen = torch.Generator().manual_seed(seed)
    W, groups = cfg["width"], cfg["norm"]["groups"]
    code = slice(W - (W // groups if groups > 1 else W // 6), W)
    w = {}
    for name, shape in tensor_shapes(cfg).items():
        t = torch.randn(*shape, generator=gen)
        if name.endswith("norm") or name.endswith("norm1"):
            t = 1 + 0.3 * t
        elif name.endswith(".act") or name.endswith("correction"):
            t = 0.5 * t
        elif name == "pos":
            t = 0.3 * t
        elif name.endswith("router"):
            t = t * (4.0 / math.sqrt(shape[-1]))
            t[:, :code.start] = 0
        elif name != "embed":
            t = t / math.sqrt(shape[-1])
        if name == "embed":
            t[:, code] = torch.sign(t[:, code])
        elif name == "pos":
            t[:, code] = 0
        elif name.endswith("norm1"):
            t[code] = 1
        elif name.endswith(".o") or name.endswith(".down"):
            t[code] = 0
        w[name] = t.bfloat16().float()
    return w
