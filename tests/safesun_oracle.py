"""Plain float64 oracle of the Safesun design: one slow function per
mechanism, written from the equations, sharing no code with the product
path. Weights come in as a dict name -> tensor under the design's
checkpoint names; the config is the config.json dict.

Notation: h is a sublayer's input [T, C]; matrices are stored [out, in];
positions count from 0.
"""

import math

import torch

F64 = torch.float64


# Where the product path may hold bfloat16 (normed sublayer inputs, projection
# outputs, cached rows, gated heads and activated feed-forwards before the
# output projection) the oracle can round too: the difference to the unrounded
# run shows how far rounding alone moves a position. Off by default.
_ROUND = [None]


class rounding:
    """with rounding(fn): every low-precision point applies fn."""

    def __init__(self, fn):
        self.fn = fn

    def __enter__(self):
        _ROUND[0] = self.fn

    def __exit__(self, *a):
        _ROUND[0] = None


def lowp(x):
    return x if _ROUND[0] is None else _ROUND[0](x)


def proj(x, w):
    return lowp(x @ w.T)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, w, eps):
    """RMS norm whose weight is stored as its distance from one."""
    return unit_rms(x, eps) * (1.0 + w)


def frequencies(rot):
    """(frequency per pair, factor on cos and sin) of a config's `rot`."""
    n, base, sc = rot["dims"], rot["base"], rot.get("scaling")
    f = [base ** (-2.0 * i / n) for i in range(n // 2)]
    if not sc:
        return f, 1.0

    def dim(turns):      # the pair (as a dimension) that makes `turns` turns over `original`
        return n * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(dim(sc["fast"])), 0)
    hi = min(math.ceil(dim(sc["slow"])), n - 1)
    out = []
    for i in range(n // 2):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f[i] / sc["factor"] * ramp + f[i] * (1.0 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, rot, first=0):
    """x [T, heads, dim] at positions first, first + 1, ...: dimension i pairs
    with i + dims/2; dimensions from rot.dims on pass."""
    if not rot or not rot.get("dims"):
        return x
    half = rot["dims"] // 2
    f, m = frequencies(rot)
    a = torch.arange(first, first + x.shape[0], dtype=F64)[:, None] * torch.tensor(f, dtype=F64)
    c, s = m * torch.cos(a)[:, None, :], m * torch.sin(a)[:, None, :]
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], -1)


def sees(i, j, mask):
    """Whether position i sees key j."""
    if j > i:
        return False
    size = (mask or {}).get("size")
    return size is None or i - j < size or j < (mask.get("keep_first") or 0)


def heads_softmax(q, k, v, scale, mask, plus_one, past=0):
    """q [n, H, D] at positions past .., k [past + n, G, D], v [.., G, Dv]."""
    n, H, _ = q.shape
    G, total = k.shape[1], past + q.shape[0]
    hidden = torch.tensor([[not sees(past + r, j, mask) for j in range(total)] for r in range(n)])
    out = torch.zeros(n, H, v.shape[-1], dtype=F64)
    for hh in range(H):
        g = hh // (H // G)
        s = ((q[:, hh] @ k[:, g].T) * scale).masked_fill(hidden, -math.inf)
        top = s.max(1, keepdim=True).values
        z = torch.exp(s - top).sum(1, keepdim=True)
        if plus_one:
            z = z + torch.exp(-top)
        out[:, hh] = (torch.exp(s - top) / z) @ v[:, g]
    return out


def mixer(h, W, p, kind, m, eps, first_values):
    """first_values: list that holds the first value-mixing layer's values once
    that layer has run."""
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    biased = kind == "attention_2"

    def part(name, heads, dim):
        y = proj(h, W[p + name])
        if biased:
            y = y + W[p + name + ".b"]
        return y.reshape(T, heads, dim)

    q, k, v = part("q", H, D), part("k", G, D), part("v", G, Dv)
    rot = m.get("rot")
    if kind == "attention":
        q = unit_rms(q, eps) * W[p + "q.norm"]
        k = unit_rms(k, eps) * W[p + "k.norm"]
        q, k = rotate(q, rot), rotate(k, rot)
    else:
        q, k = rotate(q, rot), rotate(k, rot)
        q, k = unit_rms(q, eps), unit_rms(k, eps)
    if m.get("v_mix"):
        if first_values:
            lam = W[p + "vmix"].reshape(())
            v = (1.0 - lam) * v + lam * first_values[0]
        else:
            first_values.append(v)
    out = heads_softmax(lowp(q), lowp(k), lowp(v), m["scale"], m.get("mask"), biased)
    gated = out.reshape(T, H * Dv) * sigmoid(proj(h, W[p + "g"]))
    return lowp(gated) @ W[p + "o"].T


def ff(h, W, p):
    return lowp(silu(proj(h, W[p + "gate"])) * proj(h, W[p + "up"])) @ W[p + "down"].T


def forward(cfg, W, tokens, layers_out=None):
    """Logits [T, vocab] of one whole sequence; layers_out collects the
    residual after every layer."""
    W = {k: v.to(F64) for k, v in W.items()}
    eps = cfg["norm"]["eps"]
    x = norm(W["embed"][torch.tensor(tokens)], W["embed.norm"], eps)
    first_values = []
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        y = mixer(lowp(norm(x, W[p + "norm1"], eps)), W, p + "mix.", L["type"], L["mixer"], eps,
                  first_values)
        if L.get("mlp") is not None:
            y = y + ff(lowp(norm(x, W[p + "norm2"], eps)), W, p + "mlp.")
        x = x + lowp(y)
        if layers_out is not None:
            layers_out.append(x)
    return proj(lowp(norm(x, W["final.norm"], eps)), W["embed"])


def greedy(cfg, W, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(cfg, W, toks)[-1].argmax()))
    return toks[len(prompt):]


def random_weights(cfg, seed=0):
    """Random tensors under the checkpoint's names for a config dictionary."""
    g = torch.Generator().manual_seed(seed)
    C, V = cfg["width"], cfg["vocab"]
    rn = lambda *s, std=1.0: torch.randn(*s, generator=g) * std   # noqa: E731
    W = {"embed": rn(V, C), "embed.norm": 0.2 * rn(C), "final.norm": 0.2 * rn(C)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", layer["mixer"]
        H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        W[f"l{i}.norm1"] = 0.2 * rn(C)
        for nm, n in (("q", H * D), ("k", G * D), ("v", G * Dv)):
            W[p + nm] = rn(n, C, std=C ** -0.5)
            if layer["type"] == "attention_2":
                W[p + nm + ".b"] = 0.3 * rn(n)
        if layer["type"] == "attention":
            W[p + "q.norm"] = 1.0 + 0.2 * rn(D)
            W[p + "k.norm"] = 1.0 + 0.2 * rn(D)
        if m.get("v_mix"):
            W[p + "vmix"] = (0.5 + 0.2 * rn(1)).reshape(())
        W[p + "g"] = rn(H * Dv, C, std=1.5 * C ** -0.5)
        W[p + "o"] = rn(C, H * Dv, std=2.0 * (H * Dv) ** -0.5)
        if layer.get("mlp") is not None:
            n = layer["mlp"]["ff"]
            W[f"l{i}.norm2"] = 0.2 * rn(C)
            W[f"l{i}.mlp.gate"] = rn(n, C, std=C ** -0.5)
            W[f"l{i}.mlp.up"] = rn(n, C, std=C ** -0.5)
            W[f"l{i}.mlp.down"] = rn(C, n, std=1.5 * n ** -0.5)
    return W
