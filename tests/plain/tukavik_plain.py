"""Plain implementation of the Tukavik decoder in float64, whole sequences only: one function a
mechanism, written from the equations, sharing no code with ``lockstep_amd``.  ``weights`` maps tensor
names to CPU tensors (any float dtype).

Notation: T tokens at positions 0 .. T-1, width W, H heads, query/key size d, value size e, latent rank R,
n layers.  All functions take and return float64."""

from __future__ import annotations

import math

import torch

F64 = torch.float64


def position_vectors(n, width):
    """[n, W]: at position p, element 2i is sin(p f_i) and element 2i + 1 is cos(p f_i), f_i = 10000^(-2i/W)."""
    out = torch.zeros((n, width), dtype=F64)
    for e in range(width):
        f = 10000.0 ** (-2.0 * (e // 2) / width)
        for p in range(n):
            out[p, e] = math.sin(p * f) if e % 2 == 0 else math.cos(p * f)
    return out


def layer_norm(x, weight, eps):
    """(x - mean) / sqrt(mean of squared deviations + eps) * w over the last axis."""
    d = x - x.mean(dim=-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(dim=-1, keepdim=True) + eps) * weight


def rms_norm(x, weight, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * weight


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def softplus(z):
    return torch.where(z > 30.0, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def xielu(z, p, q):
    """softplus(p) z^2 + z/2 above zero, (1/2 + softplus(q)) (e^z - 1 - z) + z/2 elsewhere."""
    low = torch.clamp(z, max=0.0)
    return torch.where(z > 0, softplus(p) * z * z, (0.5 + softplus(q)) * (torch.expm1(low) - low)) + 0.5 * z


def gated_average(z, u):
    """S_t = (1 - z_t) S_(t-1) + z_t c_t element by element from S = 0, c = u + 1/2 where u >= 0, else
    sigmoid(u).  z, u [T, w]; returns every S_t."""
    c = torch.where(u >= 0, u + 0.5, sigmoid(u))
    S = torch.zeros(z.shape[1], dtype=F64)
    out = []
    for t in range(z.shape[0]):
        S = (1.0 - z[t]) * S + z[t] * c[t]
        out.append(S)
    return torch.stack(out)


def causal_attention(q, k, v, scale):
    """One head: q, k [T, d], v [T, e]; softmax of scale q k^T over the keys j <= i."""
    n = q.shape[0]
    s = (q @ k.T) * scale
    s = s.masked_fill(~torch.tril(torch.ones((n, n), dtype=torch.bool)), -math.inf)
    p = torch.exp(s - s.max(dim=-1, keepdim=True).values)
    return (p / p.sum(dim=-1, keepdim=True)) @ v


def depth_average(results, shares):
    """sum_j shares[j] results[j]."""
    out = torch.zeros_like(results[0])
    for a, x in zip(shares, results):
        out = out + a * x
    return out


class PlainTukavik:
    def __init__(self, raw, tensors):
        self.raw = raw
        self.w = {name: t.to(F64) for name, t in tensors.items()}
        self.eps = float(raw["norm"]["eps"])

    def latent(self, i, h):
        """The latent [T, R] of layer ``i`` for its mixer's input ``h``."""
        return rms_norm(h @ self.w[f"l{i}.mix.dkv"].T, self.w[f"l{i}.mix.dkv.norm"], self.eps)

    def attention(self, i, m, h, c):
        w, p = self.w, f"l{i}.mix"
        n, heads, d, e = h.shape[0], m["heads"], m["dim"], m["vdim"]
        if f"{p}.dq" in w:
            q = rms_norm(h @ w[f"{p}.dq"].T, w[f"{p}.dq.norm"], self.eps) @ w[f"{p}.uq"].T
        else:
            q = h @ w[f"{p}.q"].T
        q, k = q.view(n, heads, d), (c @ w[f"{p}.uk"].T).view(n, heads, d)
        v = (c @ w[f"{p}.uv"].T).view(n, heads, e)
        out = [causal_attention(q[:, a], k[:, a], v[:, a], float(m["scale"])) for a in range(heads)]
        return torch.cat(out, dim=1) @ w[f"{p}.o"].T

    def recurrence(self, i, h):
        w, p = self.w, f"l{i}.mix"
        z = sigmoid(h @ w[f"{p}.z"].T + w[f"{p}.z.b"])
        S = gated_average(z, h @ w[f"{p}.x"].T + w[f"{p}.x.b"])
        g = h @ w[f"{p}.g"].T
        return (S * (g * sigmoid(g))) @ w[f"{p}.o"].T

    def feed_forward(self, i, h):
        w, p = self.w, f"l{i}.mlp"
        return xielu(h @ w[f"{p}.up"].T, w[f"{p}.act"][0], w[f"{p}.act"][1]) @ w[f"{p}.down"].T

    def run(self, tokens):
        """(logits [T, vocab], the stream behind every layer and its depth average [n, T, W])."""
        w, eps = self.w, self.eps
        tokens = torch.as_tensor(tokens, dtype=torch.long)
        x = w["embed"][tokens] + position_vectors(len(tokens), self.raw["width"])
        results, latents, after = [x], {}, []
        for i, layer in enumerate(self.raw["layers"]):
            norm = lambda name, y: layer_norm(y, w[f"l{i}.{name}"], eps)  # noqa: E731, B023
            h = norm("norm1", x)
            m = layer["mixer"]
            if layer["type"] == "mingru":
                y = self.recurrence(i, h)
            else:
                source = m.get("kv_from")
                if source is None:
                    latents[i] = self.latent(i, h)
                y = self.attention(i, m, h, latents[i if source is None else source])
            x = x + norm("norm1b", y)
            if layer.get("mlp") is not None:
                x = x + norm("norm2b", self.feed_forward(i, norm("norm2", x)))
            results.append(x)
            x = depth_average(results, w[f"l{i}.dwa"])
            after.append(x)
        logits = layer_norm(x, w["final.norm"], eps) @ w["embed"].T
        return logits, torch.stack(after)

    def forward(self, tokens):
        return self.run(tokens)[0]

    def generate_greedy(self, prompt, n):
        tokens = list(prompt)
        for _ in range(n):
            tokens.append(int(self.forward(tokens)[-1].argmax()))
        return tokens[len(prompt):]
