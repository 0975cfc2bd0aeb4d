"""Plain, slow Risepel forward pass: the oracle of the Risepel tests.

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


def zero_norm(x, weight, eps):
    """RMS norm whose weight is stored as its distance from one."""
    return rms(x, eps) * (1 + weight)


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


# -- gated linear attention -------------------------------------------------

def decays(h, w, pre, mx):
    """Per token, head and key channel: sigmoid(z)^(1/tau), [T, heads, dim]."""
    z = (h @ w[pre + "a1"].T) @ w[pre + "a2"].T + w[pre + "a2.b"]
    log = torch.nn.functional.logsigmoid(z) / mx["tau"]
    return torch.exp(log).reshape(h.shape[0], mx["heads"], mx["dim"])


def recurrence(q, k, v, a, state=None):
    """S <- diag(a_t) S + k_t v_t^T, o_t = S^T q_t, token by token.
    q, k, a [T, H, dim], v [T, H, vdim] -> o [T, H, vdim], last state."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype) if state is None else state
    out = []
    for t in range(T):
        S = a[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def gla(h, w, pre, mx, eps):
    T, H, D, V = h.shape[0], mx["heads"], mx["dim"], mx["vdim"]
    q = (h @ w[pre + "q"].T).reshape(T, H, D) * D ** -0.5
    k = (h @ w[pre + "k"].T).reshape(T, H, D)
    v = (h @ w[pre + "v"].T).reshape(T, H, V)
    o, _ = recurrence(q, k, v, decays(h, w, pre, mx))
    o = (rms(o, eps) * w[pre + "norm"]).reshape(T, H * V)
    return (o * silu(h @ w[pre + "g"].T)) @ w[pre + "o"].T


# -- latent attention -------------------------------------------------------

def rotate(x, base, dims, first=0):
    """Rotary positions on the last axis; x [T, ..., >= dims], token t at
    position first + t. Dimension i turns with i + dims / 2."""
    half = dims // 2
    T = x.shape[0]
    pos = torch.arange(first, first + T, dtype=torch.float64)
    f = base ** (-2.0 * torch.arange(half, dtype=torch.float64) / dims)
    ang = (pos[:, None] * f).reshape(T, *[1] * (x.dim() - 2), half)
    c, s = torch.cos(ang).to(x.dtype), torch.sin(ang).to(x.dtype)
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], -1)


def latent(h, w, pre, mx, eps):
    """What a token leaves in the cache: normed latent [T, kv_rank] and the
    rotated key part all heads share [T, rot_dim]."""
    y = h @ w[pre + "dkv"].T
    R = mx["kv_rank"]
    return (rms(y[:, :R], eps) * w[pre + "dkv.norm"],
            rotate(y[:, R:], mx["rot"]["base"], mx["rot"]["dims"]))


def visible(T, size):
    """[T, T] bool: query i (row) sees key j (column)."""
    d = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    return (d >= 0) & (d < size) if size else d >= 0


def attend(q, k, v, scale, size, sink):
    """q, k [T, H, dim], v [T, H, vdim], sink [H] -> [T, H, vdim]. The sink
    is one more unscaled score without a value."""
    T, H, _ = q.shape
    see = visible(T, size)
    out = torch.empty(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        s = ((q[:, h] @ k[:, h].T) * scale).masked_fill(~see, -math.inf)
        s = torch.cat([s, sink[h].expand(T, 1)], 1)
        out[:, h] = torch.softmax(s, -1)[:, :T] @ v[:, h]
    return out


def latent_attention(h, w, pre, mx, eps, kv):
    T, H, D = h.shape[0], mx["heads"], mx["dim"]
    cq = rms(h @ w[pre + "dq"].T, eps) * w[pre + "dq.norm"]
    q = (cq @ w[pre + "uq"].T).reshape(T, H, D + mx["rot_dim"])
    rot = mx["rot"]
    q = torch.cat([q[..., :D], rotate(q[..., D:], rot["base"], rot["dims"])], -1)
    c, kr = kv
    k = torch.cat([(c @ w[pre + "uk"].T).reshape(T, H, D),
                   kr[:, None].expand(T, H, kr.shape[1])], -1)
    v = (c @ w[pre + "uv"].T).reshape(T, H, mx["vdim"])
    o = attend(q, k, v, mx["scale"], (mx.get("mask") or {}).get("size"),
               w[pre + "sink"]).reshape(T, -1)
    return (o * sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T


# -- feed-forward and model -------------------------------------------------

def clamped_glu(gate, up, limit):
    g = gate.clamp(max=limit)
    u = up.clamp(-limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1)


def dense_mlp(h, w, pre, mlp):
    lin = lambda x, n: x @ w[pre + n].T + w[pre + n + ".b"]
    return lin(clamped_glu(lin(h, "gate"), lin(h, "up"), mlp["limit"]), "down")


def softcap(z, cap):
    return cap * torch.tanh(z / cap)


def forward(tokens, w, cfg, collect=None):
    """Logits [T, vocab] of one sequence; collect gets x after every layer."""
    eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
    x = w["embed"][tokens]
    kvs = []
    for i, layer in enumerate(cfg["layers"]):
        mx, mlp, p = layer["mixer"], layer["mlp"], f"l{i}."
        kvs.append(None)
        if layer["type"] == "gla":
            y = gla(x, w, p + "mix.", mx, eps)
        else:
            src = mx.get("kv_from")
            kvs[i] = (kvs[src] if src is not None
                      else latent(x, w, p + "mix.", mx, eps))
            y = latent_attention(x, w, p + "mix.", mx, eps, kvs[i])
        x = zero_norm(alpha * x + y, w[p + "norm1"], eps)
        if mlp is not None:
            x = zero_norm(alpha * x + dense_mlp(x, w, p + "mlp.", mlp),
                          w[p + "norm2"], eps)
        if collect is not None:
            collect.append(x)
    y = zero_norm(x, w["final.norm"], eps) @ w["head"].T
    return softcap(y, cfg["logit_softcap"])


# ---------------------------------------------------------------------------
# small random models
# ---------------------------------------------------------------------------

def tensor_shapes(cfg, rank=lambda layer: 3 + 4 * layer):
    """rank(layer): rows of a recurrent layer's decay projection, which the
    configuration does not name."""
    W = cfg["width"]
    s = {"embed": (cfg["vocab"], W), "final.norm": (W,), "head": (cfg["vocab"], W)}
    for i, layer in enumerate(cfg["layers"]):
        mx, mlp, p = layer["mixer"], layer["mlp"], f"l{i}."
        H, D, V = mx["heads"], mx["dim"], mx["vdim"]
        s[p + "norm1"] = (W,)
        m = p + "mix."
        s[m + "g"], s[m + "o"] = (H * V, W), (W, H * V)
        if layer["type"] == "gla":
            s[m + "q"] = s[m + "k"] = (H * D, W)
            s[m + "v"], s[m + "norm"] = (H * V, W), (V,)
            s[m + "a1"], s[m + "a2"] = (rank(i), W), (H * D, rank(i))
            s[m + "a2.b"] = (H * D,)
        else:
            Q, R, E = mx["q_rank"], mx["kv_rank"], mx["rot_dim"]
            s[m + "dq"], s[m + "dq.norm"] = (Q, W), (Q,)
            s[m + "uq"] = (H * (D + E), Q)
            s[m + "uk"], s[m + "uv"], s[m + "sink"] = (H * D, R), (H * V, R), (H,)
            if mx.get("kv_from") is None:
                s[m + "dkv"], s[m + "dkv.norm"] = (R + E, W), (R,)
        if mlp is not None:
            F = mlp["ff"]
            s[p + "norm2"] = (W,)
            for n in ("gate", "up"):
                s[p + f"mlp.{n}"], s[p + f"mlp.{n}.b"] = (F, W), (F,)
            s[p + "mlp.down"], s[p + "mlp.down.b"] = (W, F), (W,)
    return s


def random_weights(cfg, seed=0, **kw):
    """bf16-representable float32 weights of a lively scale: sharp attention,
    decays from a few tokens to hundreds, logits that meet their cap."""
    gen = torch.Generator().manual_seed(seed)
    w = {}
    for name, shape in tensor_shapes(cfg, **kw).items():
        t = torch.randn(*shape, generator=gen)
        last = name.rsplit(".", 1)[-1]
        if name.endswith(("norm1", "norm2", "final.norm")):
            t = 0.2 * t
        elif last == "norm":
            t = 1 + 0.2 * t
        elif last == "sink":
            t = 1 + t
        elif name.endswith("a2.b"):
            t = 1.5 + 1.5 * t
        elif last == "b":
            t = 0.2 * t
        elif name != "embed":
            t = t / math.sqrt(shape[-1])
            if last in ("uq", "uk"):
                t = 1.5 * t
            elif last == "head":
                t = 0.6 * cfg["logit_softcap"] * t
        w[name] = t.bfloat16().float()
    return w
