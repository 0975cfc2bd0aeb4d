"""Plain, slow Vumedra forward pass: the oracle of the Vumedra tests.

One function per mechanism, straight from the equations, whole sequences at a
time and token by token where the equation is a recurrence; no cache, no
batching, no kernels. It shares no code with bloombee_amd (only torch) and
computes in the dtype of the weights it is given; the tests pass float64.

`w` is a dict {tensor name: tensor}, `cfg` the model's configuration dict.
"""
import math

import torch


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def gelu(z):
    """The tanh form."""
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi)
                                     * (z + 0.044715 * z ** 3)))


# -- embedding ----------------------------------------------------------------

def pair_rows(ids, big):
    """Row of the pair table for every token; the first token has no
    predecessor and takes the last row."""
    prev = torch.cat([ids.new_zeros(1), ids[:-1]])
    rows = (prev * big["mul_prev"] + ids * big["mul_cur"]) % big["buckets"]
    rows[0] = big["buckets"]
    return rows


def sinusoid(first, T, width):
    """[T, width] float64: even entries sines, odd ones cosines."""
    p = torch.arange(first, first + T, dtype=torch.float64)[:, None]
    i = torch.arange((width + 1) // 2, dtype=torch.float64)
    ang = p * torch.pow(torch.tensor(10000.0, dtype=torch.float64),
                        -2 * i / width)
    return torch.stack([torch.sin(ang), torch.cos(ang)], -1).reshape(
        T, -1)[:, :width]


def embed(ids, w, cfg):
    e = w["embed"]
    return (e[ids] + w["bigram"][pair_rows(ids, cfg["embedding"]["bigram"])]
            + sinusoid(0, ids.numel(), cfg["width"]).to(e.dtype))


# -- attention ----------------------------------------------------------------

def temperature(T, qt, first=0):
    """[T] factor of the queries."""
    if not qt:
        return torch.ones(T, dtype=torch.float64)
    p = torch.arange(first, first + T, dtype=torch.float64)
    return 1 + qt["coef"] * torch.log(torch.floor((p + 1) / qt["every"]) + 1)


def sink_softmax(s):
    """exp(s_j) / (1 + sum exp(s_j)) over the last axis."""
    m = s.max(-1, keepdim=True).values.clamp(min=0)
    e = torch.exp(s - m)
    return e / (torch.exp(-m) + e.sum(-1, keepdim=True))


def attend(q, k, v, scale):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] -> [T, H, vdim]."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    later = torch.arange(T)[None, :] > torch.arange(T)[:, None]
    out = torch.empty(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        s = (q[:, h] @ k[:, h // per].T) * scale
        out[:, h] = sink_softmax(s.masked_fill(later, -math.inf)) @ v[:, h // per]
    return out


def attention(h, w, pre, mx, eps):
    T, H, G = h.shape[0], mx["heads"], mx["kv_heads"]

    def proj(n):
        return h @ w[pre + n].T + w[pre + n + ".b"]

    q = rms(proj("q").reshape(T, H, mx["dim"]), eps) * w[pre + "q.norm"]
    k = rms(proj("k").reshape(T, G, mx["dim"]), eps) * w[pre + "k.norm"]
    v = proj("v").reshape(T, G, mx["vdim"])
    q = q * temperature(T, mx.get("q_temp")).to(q.dtype)[:, None, None]
    o = attend(q, k, v, mx["scale"])
    return o.reshape(T, -1) @ w[pre + "o"].T


# -- matrix memory ------------------------------------------------------------

def capped(z, cap):
    return cap * torch.tanh(z / cap)


def memory(q, k, v, i, f, state=None):
    """Token by token. q, k [T, H, dim], v [T, H, vdim], i, f [T, H] log gates
    -> o [T, H, vdim], last (S, n, m)."""
    T, H, D = q.shape
    if state is None:
        state = (q.new_zeros(H, D, v.shape[2]), q.new_zeros(H, D),
                 q.new_zeros(H))
    S, n, m = state
    out = []
    for t in range(T):
        new = torch.maximum(f[t] + m, i[t])
        keep, add = torch.exp(f[t] + m - new), torch.exp(i[t] - new)
        m = new
        S = (keep[:, None, None] * S
             + add[:, None, None] * k[t][:, :, None] * v[t][:, None, :])
        n = keep[:, None] * n + add[:, None] * k[t]
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out.append((S * q[t][:, :, None]).sum(1) / den[:, None])
    return torch.stack(out), (S, n, m)


def mlstm(h, w, pre, mx, eps):
    T, H, D, V = h.shape[0], mx["heads"], mx["dim"], mx["vdim"]
    q = (h @ w[pre + "q"].T).reshape(T, H, D) * D ** -0.5
    k = (h @ w[pre + "k"].T).reshape(T, H, D)
    v = (h @ w[pre + "v"].T).reshape(T, H, V)
    i = capped(h @ w[pre + "i"].T + w[pre + "i.b"], mx["gate_cap"])
    f = -softplus(-capped(h @ w[pre + "f"].T + w[pre + "f.b"], mx["gate_cap"]))
    o, _ = memory(q, k, v, i, f)
    o = rms(o, eps).reshape(T, H * V) * w[pre + "norm"]
    return (o * sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T


# -- gated linear recurrent unit ---------------------------------------------

def causal_conv(x, taps, bias):
    """x [T, C], taps [C, K], the last one is the current token's."""
    K = taps.shape[1]
    past = torch.cat([x.new_zeros(K - 1, x.shape[1]), x])
    y = torch.zeros_like(x)
    for j in range(K):
        y = y + past[j:j + x.shape[0]] * taps[:, j]
    return y + bias


def block_gate(u, a, b):
    """u [T, C] in a.shape[0] equal parts, each through its square matrix."""
    B, D = b.shape
    parts = u.reshape(u.shape[0], B, D)
    z = torch.stack([parts[:, j] @ a[j].T + b[j] for j in range(B)], 1)
    return sigmoid(z).reshape(u.shape)


def unit(u, r, i, lam, S=None):
    """Token by token: [T, C] states."""
    log_a = -8 * r * softplus(lam)
    a = torch.exp(log_a)
    x = torch.sqrt(-torch.expm1(2 * log_a)) * i * u
    S = torch.zeros_like(u[0]) if S is None else S
    out = []
    for t in range(u.shape[0]):
        S = a[t] * S + x[t]
        out.append(S)
    return torch.stack(out)


def rglru(h, w, pre, mx, eps):
    y = gelu(h @ w[pre + "y"].T + w[pre + "y.b"])
    u = causal_conv(h @ w[pre + "x"].T + w[pre + "x.b"], w[pre + "conv"],
                    w[pre + "conv.b"])
    r = block_gate(u, w[pre + "ra"], w[pre + "ra.b"])
    i = block_gate(u, w[pre + "ri"], w[pre + "ri.b"])
    return (unit(u, r, i, w[pre + "lam"]) * y) @ w[pre + "o"].T


MIXERS = {"attention": attention, "mlstm": mlstm, "rglru": rglru}


# -- feed-forwards ------------------------------------------------------------

def dense(h, w, pre):
    g = h @ w[pre + "gate"].T
    return (g * sigmoid(g) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def expert(h, w, pre):
    return torch.relu(h @ w[pre + "up"].T) ** 2 @ w[pre + "down"].T


def moe(h, w, pre, mlp):
    s = sigmoid(h @ w[pre + "router"].T)
    best = torch.topk(s, mlp["router"]["top"], -1).indices
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e in best[t].tolist():
            y[t] += expert(s[t, e] * h[t], w, f"{pre}e{e}.")
    if mlp.get("shared"):
        y = y + expert(h, w, pre + "shared.")
    return y


# -- model --------------------------------------------------------------------

def layer(x, w, i, cfg):
    lay, eps, p = cfg["layers"][i], cfg["norm"]["eps"], f"l{i}."
    y = MIXERS[lay["type"]](rms(x, eps) * w[p + "norm1"], w, p + "mix.",
                            lay["mixer"], eps)
    x = x + rms(y, eps) * w[p + "norm1b"]
    mlp = lay.get("mlp")
    if mlp:
        h = rms(x, eps) * w[p + "norm2"]
        y = (dense(h, w, p + "mlp.") if mlp["kind"] == "dense"
             else moe(h, w, p + "mlp.", mlp))
        x = x + rms(y, eps) * w[p + "norm2b"]
    return x


def hidden_states(ids, w, cfg):
    """Residual after every layer, [layers, T, width]."""
    x = embed(ids, w, cfg)
    out = []
    for i in range(len(cfg["layers"])):
        x = layer(x, w, i, cfg)
        out.append(x)
    return torch.stack(out)


def forward(ids, w, cfg):
    x = hidden_states(ids, w, cfg)[-1]
    return (rms(x, cfg["norm"]["eps"]) * w["final.norm"]) @ w["head"].T


# -- random models ------------------------------------------------------------

def random_weights(cfg, seed=0):
    """bf16-representable float32 weights under the checkpoint's names."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]
    w = {}

    def put(name, *shape, std=None, mean=0.0):
        std = std if std is not None else shape[-1] ** -0.5
        w[name] = (mean + std * torch.randn(shape, generator=g)).bfloat16().float()

    put("embed", V, W, std=1.0)
    put("bigram", cfg["embedding"]["bigram"]["buckets"] + 1, W, std=1.0)
    for i, lay in enumerate(cfg["layers"]):
        p, mx, mlp = f"l{i}.", lay["mixer"], lay.get("mlp")
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if mlp else ()):
            put(p + n, std=0.2, mean=1.0)
        m = p + "mix."
        if lay["type"] == "attention":
            H, G, D, E = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
            for n, rows in (("q", H * D), ("k", G * D), ("v", G * E)):
                put(m + n, rows, W)
                put(m + n + ".b", rows, std=0.3)
            put(m + "q.norm", D, std=0.2, mean=1.5)
            put(m + "k.norm", D, std=0.2, mean=1.5)
            put(m + "o", W, H * E)
        elif lay["type"] == "mlstm":
            H, D, E = mx["heads"], mx["dim"], mx["vdim"]
            for n, rows in (("q", H * D), ("k", H * D), ("v", H * E),
                            ("g", H * E)):
                put(m + n, rows, W)
            put(m + "o", W, H * E)
            put(m + "norm", H * E, std=0.2, mean=1.0)
            # gates on both sides of the cap, forgetting fast and slowly
            for n, mean in (("i", 0.0), ("f", 3.0)):
                put(m + n, H, W, std=3 * W ** -0.5)
                put(m + n + ".b", H, std=2.0, mean=mean)
        else:
            C, B, K = mx["width"], mx["blocks"], mx["conv"]
            for n in ("y", "x"):
                put(m + n, C, W)
                put(m + n + ".b", C, std=0.3)
            put(m + "conv", C, K, std=0.5)
            put(m + "conv.b", C, std=0.3)
            for n in ("ra", "ri"):
                put(m + n, B, C // B, C // B)
                put(m + n + ".b", B, C // B, std=1.0)
            put(m + "lam", C, std=2.0, mean=-4.0)
            put(m + "o", W, C)
        if not mlp:
            continue
        m = p + "mlp."
        if mlp["kind"] == "dense":
            put(m + "gate", mlp["ff"], W)
            put(m + "up", mlp["ff"], W)
            put(m + "down", W, mlp["ff"])
            continue
        put(m + "router", mlp["router"]["experts"], W, std=2 * W ** -0.5)
        experts = {f"e{e}": mlp["expert"]["ff"]
                   for e in range(mlp["router"]["experts"])}
        if mlp.get("shared"):
            experts["shared"] = mlp["shared"]["ff"]
        for n, ff in experts.items():
            put(f"{m}{n}.up", ff, W)
            put(f"{m}{n}.down", W, ff)
    put("final.norm", std=0.2, mean=1.0)
    put("head", V, W)
    return w
