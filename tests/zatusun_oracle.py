"""Plain, slow Zatusun forward pass: the oracle of the Zatusun tests.

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


def norm(x, w, eps):
    """RMS norm whose weight is stored as its distance from one."""
    return rms(x, eps) * (1 + w)


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softmax(s):
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


# -- embedding ----------------------------------------------------------------

def embed(ids, w, cfg):
    return (w["embed"][ids] * cfg["embedding"]["scale"]
            + w["pos"][torch.arange(ids.numel())])


# -- rotation -----------------------------------------------------------------

def plain_frequencies(base, dims):
    return [base ** (-2 * i / dims) for i in range(dims // 2)]


def yarn(rot):
    """Frequencies and the factor of cosine and sine."""
    base, dims, s = rot["base"], rot["dims"], rot.get("scaling")
    f = plain_frequencies(base, dims)
    if not s:
        return f, 1.0

    def dim(turns):
        return (dims * math.log(s["original"] / (2 * math.pi * turns))
                / (2 * math.log(base)))

    lo = max(math.floor(dim(s["fast"])), 0)
    hi = min(math.ceil(dim(s["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / s["factor"] * ramp + fi * (1 - ramp))
    return out, 0.1 * math.log(s["factor"]) + 1


def banded(rot):
    """Long wavelengths slowed down, short ones kept, a blend between."""
    s = rot.get("scaling")
    out = []
    for f in plain_frequencies(rot["base"], rot["dims"]):
        if s:
            l = 2 * math.pi / f
            if l > s["original"] / s["low"]:
                f = f / s["factor"]
            elif l >= s["original"] / s["high"]:
                t = (s["original"] / l - s["low"]) / (s["high"] - s["low"])
                f = (1 - t) * f / s["factor"] + t * f
        out.append(f)
    return out, 1.0


def rotate(x, freqs, factor=1.0, first=0):
    """x [T, ..., D] at positions first ..: elements 2i and 2i + 1 turn together,
    those beyond the pairs pass."""
    p = torch.arange(first, first + x.shape[0], dtype=torch.float64)
    y = x.clone()
    for i, f in enumerate(freqs):
        a = (p * f).reshape([-1] + [1] * (x.dim() - 2))
        c, s = (factor * torch.cos(a)).to(x), (factor * torch.sin(a)).to(x)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        y[..., 2 * i], y[..., 2 * i + 1] = u * c - v * s, v * c + u * s
    return y


# -- attention ----------------------------------------------------------------

def attend(q, k, v, scale, chunk=0):
    """q [T, H, D], k [T, H, D], v [T, H, V] -> [T, H, V]; with chunk, a query
    sees its own chunk of positions only."""
    T = q.shape[0]
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    if chunk:
        seen = seen & (i // chunk == j // chunk)
    out = torch.empty(T, q.shape[1], v.shape[2], dtype=q.dtype)
    for h in range(q.shape[1]):
        s = (q[:, h] @ k[:, h].T) * scale
        out[:, h] = softmax(s.masked_fill(~seen, -math.inf)) @ v[:, h]
    return out


def latent_attention(h, w, pre, mx, eps):
    T, H, D, R, V = (h.shape[0], mx["heads"], mx["dim"], mx["rot_dim"],
                     mx["vdim"])
    freqs, factor = yarn(mx["rot"])
    cq = rms(h @ w[pre + "dq"].T, eps) * w[pre + "dq.norm"]
    q = (cq @ w[pre + "uq"].T).reshape(T, H, D + R)
    q = torch.cat([q[..., :D], rotate(q[..., D:], freqs, factor)], -1)
    y = h @ w[pre + "dkv"].T
    c = rms(y[:, :mx["kv_rank"]], eps) * w[pre + "dkv.norm"]
    r = rotate(y[:, mx["kv_rank"]:], freqs, factor)
    k = torch.cat([(c @ w[pre + "uk"].T).reshape(T, H, D),
                   r[:, None].expand(T, H, R)], -1)
    v = (c @ w[pre + "uv"].T).reshape(T, H, V)
    o = attend(q, k, v, mx["scale"]).reshape(T, H * V)
    return (o * sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T


def mix_factor(w, pre, diff):
    """The second map's share."""
    return (torch.exp((w[pre + "lq1"] * w[pre + "lk1"]).sum())
            - torch.exp((w[pre + "lq2"] * w[pre + "lk2"]).sum()) + diff)


def differential(q, k, v, scale, chunk, lam, diff, eps):
    """q [T, H, 2, D], k [T, G, 2, D], v [T, G, V] -> [T, H, V]: the difference
    of two attentions over the same values, normed per head."""
    per = q.shape[1] // k.shape[1]
    v = v.repeat_interleave(per, 1)
    a = [attend(q[:, :, m], k[:, :, m].repeat_interleave(per, 1), v, scale, chunk)
         for m in range(2)]
    return rms(a[0] - lam * a[1], eps) * (1 - diff)


def attention(h, w, pre, mx, eps):
    T, H, G, D, V = (h.shape[0], mx["heads"], mx["kv_heads"], mx["dim"],
                     mx["vdim"])
    freqs, _ = banded(mx["rot"])
    q = rotate((h @ w[pre + "q"].T).reshape(T, H, 2, D), freqs)
    k = rotate((h @ w[pre + "k"].T).reshape(T, G, 2, D), freqs)
    v = (h @ w[pre + "v"].T).reshape(T, G, V)
    chunk = (mx.get("mask") or {}).get("size", 0)
    o = differential(q, k, v, mx["scale"], chunk,
                     mix_factor(w, pre, mx["diff"]), mx["diff"], eps)
    return o.reshape(T, H * V) @ w[pre + "o"].T


# -- recurrence ---------------------------------------------------------------

def forget(z, lower):
    return lower + (1 - lower) * sigmoid(z)


def scan(q, f, v, S=None):
    """Token by token: q, f [T, H, D], v [T, H, V] -> o [T, H, V], last state;
    what a channel forgets makes room for the new value."""
    if S is None:
        S = q.new_zeros(q.shape[1], q.shape[2], v.shape[2])
    out = []
    for t in range(q.shape[0]):
        S = f[t][:, :, None] * S + (1 - f[t])[:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def hgrn2(h, w, pre, mx, eps):
    T, H, D, V = h.shape[0], mx["heads"], mx["dim"], mx["vdim"]
    q = silu(h @ w[pre + "q"].T).reshape(T, H, D)
    f = forget(h @ w[pre + "f"].T + w[pre + "f.b"], w[pre + "lower"])
    v = (h @ w[pre + "v"].T).reshape(T, H, V)
    o, _ = scan(q, f.reshape(T, H, D), v)
    return (rms(o, eps) * w[pre + "norm"]).reshape(T, H * V) @ w[pre + "o"].T


MIXERS = {"latent_attention": latent_attention, "attention": attention,
          "hgrn2": hgrn2}


# -- feed-forward -------------------------------------------------------------

def clamped_glu(g, u, limit):
    g, u = g.clamp(max=limit), u.clamp(-limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1)


def expert(h, w, pre, limit):
    return clamped_glu(h @ w[pre + "gate"].T, h @ w[pre + "up"].T,
                       limit) @ w[pre + "down"].T


def choose(z, top):
    """Indices and weights of the largest logits, softmax over these alone."""
    best = torch.topk(z, top, -1)
    return best.indices, softmax(best.values)


def moe(h, w, pre, mlp):
    ids, share = choose(h @ w[pre + "router"].T, mlp["router"]["top"])
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, p in zip(ids[t].tolist(), share[t]):
            y[t] += p * expert(h[t], w, f"{pre}e{e}.", mlp["expert"]["limit"])
    return y


# -- model --------------------------------------------------------------------

def layer(x, w, i, cfg):
    lay, eps, p = cfg["layers"][i], cfg["norm"]["eps"], f"l{i}."
    x = x + MIXERS[lay["type"]](norm(x, w[p + "norm1"], eps), w, p + "mix.",
                                lay["mixer"], eps)
    if lay.get("mlp"):
        x = x + moe(norm(x, w[p + "norm2"], eps), w, p + "mlp.", lay["mlp"])
    return x


def order(cfg):
    """(layer, pass or None) of every layer run; the pass at its first layer."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    runs = [(i, None) for i in range(a)]
    for t in range(loop["times"]):
        runs += [(i, t if i == a else None) for i in range(a, b)]
    return runs + [(i, None) for i in range(b, n)]


def enter_pass(x, x0, t, w):
    return torch.cat([x, x0], -1) @ w["loop.in"].T + w["loop.step"][t]


def hidden_states(ids, w, cfg):
    """Residual after every layer run, [runs, T, width]."""
    x0 = x = embed(ids, w, cfg)
    out = []
    for i, t in order(cfg):
        if t is not None:
            x = enter_pass(x, x0, t, w)
        x = layer(x, w, i, cfg)
        out.append(x)
    return torch.stack(out)


def softcap(z, cap):
    return cap * torch.tanh(z / cap)


def head(x, w, cfg):
    z = norm(x, w["final.norm"], cfg["norm"]["eps"]) @ w["head"].T
    cap = cfg.get("logit_softcap")
    return softcap(z, cap) if cap else z


def forward(ids, w, cfg):
    return head(hidden_states(ids, w, cfg)[-1], w, cfg)


# -- random models ------------------------------------------------------------

def random_weights(cfg, seed=0):
    """bf16-representable float32 weights under the checkpoint's names."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]
    w = {}

    def put(name, *shape, std=None, mean=0.0):
        std = std if std is not None else shape[-1] ** -0.5
        w[name] = (mean + std * torch.randn(shape, generator=g)).bfloat16().float()

    put("embed", V, W, std=1 / cfg["embedding"]["scale"])
    put("pos", cfg["max_positions"], W, std=0.5)
    if cfg.get("loop"):
        put("loop.in", W, 2 * W)
        put("loop.step", cfg["loop"]["times"], W, std=0.5)
    for i, lay in enumerate(cfg["layers"]):
        p, mx, mlp = f"l{i}.", lay["mixer"], lay.get("mlp")
        H, D, E = mx["heads"], mx["dim"], mx["vdim"]
        for n in ("norm1", "norm2") if mlp else ("norm1",):
            put(p + n, W, std=0.2)
        m = p + "mix."
        put(m + "o", W, H * E)
        if lay["type"] == "latent_attention":
            R, K, Q = mx["rot_dim"], mx["kv_rank"], mx["q_rank"]
            put(m + "dq", Q, W)
            put(m + "dq.norm", Q, std=0.2, mean=1.2)
            put(m + "uq", H * (D + R), Q)
            put(m + "dkv", K + R, W)
            put(m + "dkv.norm", K, std=0.2, mean=1.2)
            put(m + "uk", H * D, K)
            put(m + "uv", H * E, K)
            put(m + "g", H * E, W)
        elif lay["type"] == "attention":
            G = mx["kv_heads"]
            put(m + "q", 2 * H * D, W)
            put(m + "k", 2 * G * D, W)
            put(m + "v", G * E, W)
            for n in ("lq1", "lk1", "lq2", "lk2"):
                put(m + n, D, std=0.6 * D ** -0.25)
        else:
            for n, rows in (("q", H * D), ("f", H * D), ("v", H * E)):
                put(m + n, rows, W)
            put(m + "f.b", H * D, std=1.5, mean=2.0)
            # lower bounds between nearly zero and nearly one
            w[m + "lower"] = (0.98 * torch.rand(H * D, generator=g)).bfloat16().float()
            put(m + "norm", E, std=0.2, mean=1.0)
        if not mlp:
            continue
        m, ff = p + "mlp.", mlp["expert"]["ff"]
        put(m + "router", mlp["router"]["experts"], W, std=2 * W ** -0.5)
        for e in range(mlp["router"]["experts"]):
            put(f"{m}e{e}.gate", ff, W)
            put(f"{m}e{e}.up", ff, W)
            put(f"{m}e{e}.down", W, ff)
    put("final.norm", W, std=0.2)
    put("head", V, W)
    return w
