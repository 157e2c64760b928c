"""Plain implementation of the Pozozen decoder in float64, whole sequences only: one function a
mechanism, written from the equations, sharing no code with ``lockstep_amd``.  ``weights`` maps tensor
names to CPU tensors (any float dtype).

Notation: T tokens at positions 0 .. T-1, width W, H heads, key size d, value size e, N rows of a state
matrix a head.  All functions take and return float64."""

from __future__ import annotations

import math

import torch

F64 = torch.float64


def layer_norm(x, weight, bias, eps):
    """(x - mean) / sqrt(mean of squared deviations + eps) * w + b over the last axis."""
    d = x - x.mean(dim=-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(dim=-1, keepdim=True) + eps) * weight + bias


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.where(z > 30.0, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def log_sigmoid(z):
    return -softplus(-z)


def window_attention(q, k, v, scale, window):
    """One head: q, k [T, d], v [T, e]; softmax of scale q k^T over the keys j with 0 <= i - j < window (None: all
    earlier ones)."""
    n = q.shape[0]
    out = torch.zeros((n, v.shape[1]), dtype=F64)
    for i in range(n):
        lo = 0 if window is None else max(0, i - window + 1)
        s = (k[lo:i + 1] @ q[i]) * scale
        p = torch.exp(s - s.max())
        out[i] = (p / p.sum()) @ v[lo:i + 1]
    return out


def causal_conv(x, taps, bias):
    """x [T, C], taps [C, M] (the last column is the current token's), zeros before the start."""
    m = taps.shape[1]
    padded = torch.cat([torch.zeros((m - 1, x.shape[1]), dtype=F64), x])
    out = torch.zeros_like(x)
    for j in range(m):
        out = out + padded[j:j + x.shape[0]] * taps[:, j]
    return out + bias


def state_space(x, b, c, dt, rate, skip):
    """One head: S <- exp(-rate dt_t) S + dt_t b_t x_t^T, y_t = S^T c_t + skip x_t.  x [T, e], b, c [T, N], dt [T]."""
    S = torch.zeros((b.shape[1], x.shape[1]), dtype=F64)
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(-rate * dt[t]) * S + dt[t] * torch.outer(b[t], x[t])
        out[t] = S.T @ c[t] + skip * x[t]
    return out


def matrix_memory(q, k, v, i, f):
    """One head of the stabilised matrix memory: q, k [T, d], v [T, e]; log input gate i and log forget gate f [T]."""
    S = torch.zeros((k.shape[1], v.shape[1]), dtype=F64)
    n = torch.zeros(k.shape[1], dtype=F64)
    m = torch.zeros((), dtype=F64)
    out = torch.zeros_like(v)
    for t in range(q.shape[0]):
        fresh = torch.maximum(f[t] + m, i[t])
        keep, write = torch.exp(f[t] + m - fresh), torch.exp(i[t] - fresh)
        S = keep * S + write * torch.outer(k[t], v[t])
        n = keep * n + write * k[t]
        m = fresh
        out[t] = (S.T @ q[t]) / (torch.maximum((n @ q[t]).abs(), torch.exp(-m)) + 1e-6)
    return out


def choose(scores, correction, top, groups, keep):
    """(indices [T, top], weights [T, top]) of the router: softmax ``scores`` [T, R] with ``correction`` [R] for the choice
    only, restricted to the ``keep`` of ``groups`` equal runs of neighbours whose best choice score is largest."""
    choice = scores + correction
    t, r = choice.shape
    best = choice.view(t, groups, r // groups).max(dim=-1).values
    kept = best.sort(dim=-1, descending=True, stable=True).indices[:, :keep]
    open_ = torch.zeros((t, groups), dtype=torch.bool).scatter_(1, kept, True).repeat_interleave(r // groups, dim=1)
    chosen = choice.masked_fill(~open_, -math.inf).sort(dim=-1, descending=True, stable=True).indices[:, :top]
    w = scores.gather(1, chosen)
    return chosen, w / (w.sum(dim=-1, keepdim=True) + 1e-20)


def read_streams(xs, take):
    return sum(a * x for a, x in zip(take, xs))


def write_streams(xs, mix, gain, y):
    return [sum(mix[s, t] * xs[s] for s in range(len(xs))) + gain[t] * y for t in range(len(xs))]


class PlainPozozen:
    def __init__(self, raw, tensors):
        self.raw = raw
        self.w = {name: t.to(F64) for name, t in tensors.items()}
        self.eps = float(raw["norm"]["eps"])
        self.m = float(raw["residual_mult"])

    def norm(self, name, x):
        return layer_norm(x, self.w[name], self.w[f"{name}.b"], self.eps)

    def attention(self, p, m, h):
        w, n, heads, g, d, e = self.w, h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        q = (h @ w[f"{p}.q"].T + w[f"{p}.q.b"]).view(n, heads, d)
        k = (h @ w[f"{p}.k"].T + w[f"{p}.k.b"]).view(n, g, d)
        v = (h @ w[f"{p}.v"].T + w[f"{p}.v.b"]).view(n, g, e)
        window = m["mask"]["size"] if m.get("mask") else None
        each = heads // g
        return torch.cat([window_attention(q[:, a], k[:, a // each], v[:, a // each], float(m["scale"]), window)
                          for a in range(heads)], dim=1) @ w[f"{p}.o"].T

    def mamba(self, p, m, h):
        w, n, heads, e, N, G = self.w, h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
        inner = heads * e
        z, conv_in, dt = torch.split(h @ w[f"{p}.in"].T, [inner, inner + 2 * G * N, heads], dim=1)
        x, b, c = torch.split(silu(causal_conv(conv_in, w[f"{p}.conv"], w[f"{p}.conv.b"])), [inner, G * N, G * N], dim=1)
        dt = softplus(dt + w[f"{p}.dt_bias"])
        x, b, c = x.view(n, heads, e), b.view(n, G, N), c.view(n, G, N)
        each = heads // G
        y = torch.cat([state_space(x[:, a], b[:, a // each], c[:, a // each], dt[:, a], torch.exp(w[f"{p}.A_log"][a]),
                                   w[f"{p}.D"][a]) for a in range(heads)], dim=1)
        y = unit_rms((y * silu(z)).view(n, m["norm_groups"], -1), self.eps).reshape(n, inner)
        return (y * w[f"{p}.norm"]) @ w[f"{p}.o"].T

    def parallel(self, p, m, h):
        return float(m["left_scale"]) * self.attention(f"{p}.left", m["left"], h) + \
            float(m["right_scale"]) * self.mamba(f"{p}.right", m["right"], h)

    def mlstm(self, p, m, h):
        w, n, heads, d, e, cap = self.w, h.shape[0], m["heads"], m["dim"], m["vdim"], float(m["gate_cap"])
        q = (h @ w[f"{p}.q"].T).view(n, heads, d) * d ** -0.5
        k = (h @ w[f"{p}.k"].T).view(n, heads, d)
        v = (h @ w[f"{p}.v"].T).view(n, heads, e)
        i = cap * torch.tanh((h @ w[f"{p}.i"].T + w[f"{p}.i.b"]) / cap)
        f = log_sigmoid(cap * torch.tanh((h @ w[f"{p}.f"].T + w[f"{p}.f.b"]) / cap))
        o = torch.cat([unit_rms(matrix_memory(q[:, a], k[:, a], v[:, a], i[:, a], f[:, a]), self.eps)
                       for a in range(heads)], dim=1)
        return (o * w[f"{p}.norm"] * sigmoid(h @ w[f"{p}.g"].T)) @ w[f"{p}.o"].T

    def gated(self, p, h):
        w = self.w
        return (silu(h @ w[f"{p}.gate"].T) * (h @ w[f"{p}.up"].T)) @ w[f"{p}.down"].T

    def experts(self, p, mlp, h):
        router = mlp["router"]
        groups = router.get("groups") or {"count": 1, "keep": 1}
        scores = torch.softmax(h @ self.w[f"{p}.router"].T, dim=-1)
        chosen, weight = choose(scores, self.w[f"{p}.correction"], router["top"], groups["count"], groups["keep"])
        out = torch.zeros_like(h)
        for t in range(h.shape[0]):
            for e, a in zip(chosen[t].tolist(), weight[t]):
                out[t] += a * (self.gated(f"{p}.e{e}", h[t]) if e < router["experts"] else h[t])
        return out + self.gated(f"{p}.shared", h) if mlp.get("shared") else out

    def order(self):
        n, loop = len(self.raw["layers"]), self.raw.get("loop")
        if not loop:
            return list(range(n))
        inside = list(range(loop["start"], loop["stop"]))
        return list(range(loop["start"])) + inside * loop["times"] + list(range(loop["stop"], n))

    def run(self, tokens):
        """(logits [T, vocab], the sum of the streams behind every run of a layer [runs, T, W])."""
        w = self.w
        x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
        s = self.raw.get("streams")
        xs = [x] * (s or 1)
        after = []
        for i in self.order():
            layer = self.raw["layers"][i]
            mixer = self.parallel if layer["type"] == "parallel" else self.mlstm
            sublayers = [("1", lambda h: mixer(f"l{i}.mix", layer["mixer"], h))]  # noqa: B023
            if layer.get("mlp"):
                sublayers.append(("2", lambda h: self.experts(f"l{i}.mlp", layer["mlp"], h)))  # noqa: B023
            for q, f in sublayers:
                if s:
                    y = f(self.norm(f"l{i}.norm{q}", read_streams(xs, w[f"l{i}.hc{q}.in"])))
                    xs = write_streams(xs, w[f"l{i}.hc{q}.mix"], self.m * w[f"l{i}.hc{q}.out"], y)
                else:
                    xs = [xs[0] + self.m * f(self.norm(f"l{i}.norm{q}", xs[0]))]
            after.append(sum(xs))
        return self.norm("final.norm", sum(xs)) @ w["head"].T, torch.stack(after)

    def forward(self, tokens):
        return self.run(tokens)[0]

    def generate_greedy(self, prompt, n):
        tokens = list(prompt)
        for _ in range(n):
            tokens.append(int(self.forward(tokens)[-1].argmax()))
        return tokens[len(prompt):]
