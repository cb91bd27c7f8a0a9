"""Plain float64 restatement of models described by a list of layers (Vadonex): one function per mechanism, one
token at a time wherever a mechanism is causal.  TEST INFRASTRUCTURE ONLY: the product never imports this, and this
imports nothing of the product.

A model is a dict: {"width", "vocab", "eps", "alpha", "layers": [...]} with, per layer,
    mixer  {"type": "latent_attention", "heads", "dim", "rot_dim", "vdim", "kv_rank", "window", "scale",
            "rot_base", "rot_dims", "kv_from" (or None)}
        or {"type": "general_delta", "heads", "dim"}
    mlp    None, {"kind": "dense"} or {"kind": "moe", "experts", "top", "shared" (bool)}
and weights a dict name -> float64 array.
"""
import math

import numpy as np


def rms_norm(x, eps, w=None):
    y = x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)
    return y if w is None else y * w


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def softplus(z):
    return math.log1p(math.exp(-abs(z))) + max(z, 0.0)


_erf = np.vectorize(math.erf)


def gelu_erf(z):
    return 0.5 * z * (1.0 + _erf(z / math.sqrt(2.0)))


def xielu(z, p, q):
    pos = softplus(p) * z * z + 0.5 * z
    zn = np.minimum(z, 0.0)
    neg = (0.5 + softplus(q)) * (np.exp(zn) - 1.0 - zn) + 0.5 * z
    return np.where(z > 0, pos, neg)


def rotate(v, pos, base, dims):
    """Interleaved pairs (2i, 2i+1) of the first `dims` entries of v turned by pos * base^(-2i/dims)."""
    out = np.array(v, dtype=np.float64)
    for i in range(dims // 2):
        a = pos * base ** (-2.0 * i / dims)
        c, s = math.cos(a), math.sin(a)
        u, w = v[..., 2 * i], v[..., 2 * i + 1]
        out[..., 2 * i] = u * c - w * s
        out[..., 2 * i + 1] = w * c + u * s
    return out


def latent_kv(m, w, pre, h, eps, pos):
    """(latent, rotated key part) of one token: what a layer caches."""
    z = w[pre + "dkv"] @ h
    c = rms_norm(z[: m["kv_rank"]], eps, w[pre + "dkv.norm"])
    return c, rotate(z[m["kv_rank"]:], pos, m["rot_base"], m["rot_dims"])


def latent_attention(m, w, pre, h, eps, pos, cacheC, cacheR):
    """One token at position pos against cached latents / rotated parts of positions 0 .. pos."""
    H, D, R, V = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    cq = rms_norm(w[pre + "dq"] @ h, eps, w[pre + "dq.norm"])
    q = (w[pre + "uq"] @ cq).reshape(H, D + R)
    qn, qr = q[:, :D], rotate(q[:, D:], pos, m["rot_base"], m["rot_dims"])
    lo = 0 if not m["window"] else max(0, pos - m["window"] + 1)
    C, Rk = np.asarray(cacheC[lo: pos + 1]), np.asarray(cacheR[lo: pos + 1])
    out = np.empty((H, V))
    for i in range(H):
        k = C @ w[pre + "uk"][i * D:(i + 1) * D].T
        v = C @ w[pre + "uv"][i * V:(i + 1) * V].T
        s = (k @ qn[i] + Rk @ qr[i]) * m["scale"]
        p = np.exp(s - s.max())
        out[i] = (p / p.sum()) @ v
    return w[pre + "o"] @ out.ravel()


def delta_update(S, decay, a, u, k, v):
    """S <- diag(decay) S - (a u)(u^T S) + k v^T, both terms from the old state; S is [key channel, value channel]."""
    return decay[:, None] * S - np.outer(a * u, u @ S) + np.outer(k, v)


def general_delta(m, w, pre, h, eps, S):
    """One token; S [heads, dim, dim] is updated in place."""
    H, D = m["heads"], m["dim"]
    r, k, v = ((w[pre + n] @ h).reshape(H, D) for n in ("r", "k", "v"))
    dec = np.exp(-math.exp(-0.5) * sigmoid(w[pre + "w2"] @ np.tanh(w[pre + "w1"] @ h) + w[pre + "w0"])).reshape(H, D)
    a = sigmoid(w[pre + "a"] @ h + w[pre + "a.b"]).reshape(H, D)
    o = np.empty((H, D))
    for i in range(H):
        u = k[i] / math.sqrt(float(k[i] @ k[i]) + 1e-6)
        S[i] = delta_update(S[i], dec[i], a[i], u, k[i], v[i])
        o[i] = S[i].T @ r[i]
    y = rms_norm(o, eps).ravel() * w[pre + "norm"] * sigmoid(w[pre + "g"] @ h)
    return w[pre + "o"] @ y


def dense_ff(w, pre, h):
    p, q = (float(t) for t in w[pre + "act"])
    return w[pre + "down"] @ xielu(w[pre + "up"] @ h, p, q)


def expert_ff(w, pre, h):
    return w[pre + "down"] @ gelu_erf(w[pre + "up"] @ h)


def route(z, top):
    """Chosen experts (largest score first, the lower index on ties) and their softmax scores over all experts."""
    s = np.exp(z - z.max())
    s /= s.sum()
    order = sorted(range(len(z)), key=lambda e: (-s[e], e))[:top]
    return order, s[order]


def moe_ff(m, w, pre, h):
    chosen, weight = route(w[pre + "router"] @ h, m["top"])
    y = np.zeros_like(h)
    for e, g in zip(chosen, weight):
        y += g * expert_ff(w, f"{pre}e{e}.", h)
    if m["shared"]:
        y += expert_ff(w, pre + "shared.", h)
    return y


class Oracle:
    """A sequence of one model: step(token) returns logits and keeps every layer's output in .trail."""

    def __init__(self, model, weights):
        self.m, self.w = model, {k: np.asarray(v, np.float64) for k, v in weights.items()}
        self.reset()

    def reset(self):
        self.pos = 0
        self.C = [[] for _ in self.m["layers"]]
        self.R = [[] for _ in self.m["layers"]]
        self.S = [np.zeros((L["mixer"]["heads"],) + (L["mixer"]["dim"],) * 2) if L["mixer"]["type"] == "general_delta" else None
                  for L in self.m["layers"]]

    def step(self, token):
        M, w, eps = self.m, self.w, self.m["eps"]
        x = w["embed"][token].copy()
        X, self.trail = [x], []
        for i, L in enumerate(M["layers"]):
            m, pre = L["mixer"], f"l{i}.mix."
            if m["type"] == "general_delta":
                y = general_delta(m, w, pre, x, eps, self.S[i])
            else:
                src = i if m["kv_from"] is None else m["kv_from"]
                if src == i:
                    c, r = latent_kv(m, w, pre, x, eps, self.pos)
                    self.C[i].append(c)
                    self.R[i].append(r)
                y = latent_attention(m, w, pre, x, eps, self.pos, self.C[src], self.R[src])
            x = rms_norm(M["alpha"] * x + y, eps, w[f"l{i}.norm1"])
            if L["mlp"] is not None:
                pre = f"l{i}.mlp."
                y = dense_ff(w, pre, x) if L["mlp"]["kind"] == "dense" else moe_ff(L["mlp"], w, pre, x)
                x = rms_norm(M["alpha"] * x + y, eps, w[f"l{i}.norm2"])
            X.append(x)
            x = sum(d * t for d, t in zip(w[f"l{i}.dwa"], X))
            self.trail.append(x)
        self.pos += 1
        return w["head"] @ rms_norm(x, eps, w["final.norm"])

    def run(self, tokens):
        return np.stack([self.step(int(t)) for t in tokens])

    def greedy(self, prompt, n):
        logits = self.run(prompt)[-1]
        out = []
        for _ in range(n):
            out.append(int(np.argmax(logits)))
            logits = self.step(out[-1])
        return out
