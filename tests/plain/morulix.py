"""A plain, slow implementation of the Morulix decoder, one function per mechanism, written from the
design's equations with torch on the CPU (64-bit by default). It shares no code with the engine: it
reads config.json and model.safetensors itself. The tests compare the engine with it.

Notation. rms(x) = x / sqrt(mean(x^2) + eps), n(x) = rms(x) (1 + w). A layer computes
x <- x + (mixer(n x) + ff(n x)), one norm for both. The mixer is one of three: a state-space mixer with a
scalar decay per head behind a short convolution ("mamba2"), grouped-query attention in a sliding window
with half-rotated heads ("attention"), or attention through a low-rank latent without positions, with a
learned sink and a gate per head ("latent_attention"). A stretch of layers may run several times in a row
with the same weights; ahead of each pass x <- W_in [x; x0] + step[t], x0 the embedded tokens. Every pass
keeps caches and states of its own.
"""

from __future__ import annotations

import json
import math
import os

import torch
from safetensors import safe_open


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x divided by its root mean square over the last dimension, eps inside the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """The layers' norm: its weight is stored around zero."""
    return unit_rms(x, eps) * (1.0 + w)


def pass_input(x: torch.Tensor, x0: torch.Tensor, w_in: torch.Tensor, step: torch.Tensor) -> torch.Tensor:
    """What a pass through the looped layers starts from: W_in [x; x0] + step."""
    return torch.cat([x, x0], dim=-1) @ w_in.T + step


def banded_frequencies(dims: int, base: float, scaling: dict | None) -> list[float]:
    """f_i = base^(-2i/dims), i < dims/2. With scaling (factor s, low, high, original L) by wavelength
    l = 2 pi / f: f if l < L/high; f/s if l > L/low; between, with m = (L/l - low)/(high - low),
    (1 - m) f/s + m f."""
    out = []
    for i in range(dims // 2):
        f = float(base) ** (-2.0 * i / dims)
        if scaling:
            s, low, high, length = (float(scaling[k]) for k in ("factor", "low", "high", "original"))
            wave = 2.0 * math.pi / f
            if wave > length / low:
                f = f / s
            elif not wave < length / high:
                m = (length / wave - low) / (high - low)
                f = (1.0 - m) * f / s + m * f
        out.append(f)
    return out


def rotate_halves(x: torch.Tensor, positions: torch.Tensor, freqs: list[float]) -> torch.Tensor:
    """x [n, heads, D]: of every head the pairs (i, i + len(freqs)) turn by position * freqs[i]; the rest pass."""
    half = len(freqs)
    out = x.clone()
    for i, f in enumerate(freqs):
        a = positions.to(torch.float64) * f
        c, s = torch.cos(a).to(x.dtype)[:, None], torch.sin(a).to(x.dtype)[:, None]
        u, v = x[:, :, i], x[:, :, i + half]
        out[:, :, i] = u * c - v * s
        out[:, :, i + half] = v * c + u * s
    return out


def softmax_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, q_positions: torch.Tensor, scale: float,
                      window: int = 0, sinks: torch.Tensor | None = None) -> torch.Tensor:
    """q [n, H, D] at `q_positions` over keys k [m, G, D], values v [m, G, V] at positions 0..m-1. Position i sees
    0 <= i - j (< window if there is one); weight_j = exp(s_j) / (sum_j' exp(s_j') [+ exp(sink_h)])."""
    n, H, _ = q.shape
    G = k.shape[1]
    gap = q_positions[:, None] - torch.arange(k.shape[0])[None, :]
    see = gap >= 0
    if window:
        see = see & (gap < window)
    out = torch.zeros(n, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].T) * scale).masked_fill(~see, float("-inf"))
        top = s.max(dim=-1, keepdim=True).values
        if sinks is not None:
            top = torch.maximum(top, sinks[h])
        e = torch.exp(s - top)
        total = e.sum(-1, keepdim=True) + (torch.exp(sinks[h] - top) if sinks is not None else 0.0)
        out[:, h] = (e / total) @ v[:, g]
    return out


def window_attention(h: torch.Tensor, positions: torch.Tensor, W: dict, m: dict, past: dict) -> torch.Tensor:
    """The "attention" mixer for the rows h at `positions`; `past` holds the keys and values so far."""
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    n = h.shape[0]
    rot = m.get("rot") or {}
    freqs = banded_frequencies(int(rot["dims"]), rot["base"], rot.get("scaling")) if rot.get("dims") else []
    q = rotate_halves((h @ W["q"].T).reshape(n, H, D), positions, freqs)
    k = rotate_halves((h @ W["k"].T).reshape(n, G, D), positions, freqs)
    v = (h @ W["v"].T).reshape(n, G, V)
    past["k"] = torch.cat([past["k"], k]) if "k" in past else k
    past["v"] = torch.cat([past["v"], v]) if "v" in past else v
    size = int(m["mask"]["size"]) if m.get("mask") else 0
    o = softmax_attention(q, past["k"], past["v"], positions, float(m["scale"]), window=size)
    return o.reshape(n, H * V) @ W["o"].T


def latent_attention(h: torch.Tensor, positions: torch.Tensor, W: dict, m: dict, eps: float, past: dict) -> torch.Tensor:
    """The "latent_attention" mixer; `past` holds the latents so far. Keys and values of all heads are
    up-projections of the latent; nothing turns; every position before sees; the gate is a number per head."""
    H, D, V = m["heads"], m["dim"], m["vdim"]
    n = h.shape[0]
    q = (h @ W["q"].T).reshape(n, H, D)
    c = unit_rms(h @ W["dkv"].T, eps) * W["dkv.norm"]
    past["c"] = torch.cat([past["c"], c]) if "c" in past else c
    k = (past["c"] @ W["uk"].T).reshape(-1, H, D)
    v = (past["c"] @ W["uv"].T).reshape(-1, H, V)
    o = softmax_attention(q, k, v, positions, float(m["scale"]), sinks=W["sink"])
    o = o * torch.sigmoid(h @ W["g"].T)[:, :, None]
    return o.reshape(n, H * V) @ W["o"].T


def convolve(u: torch.Tensor, w: torch.Tensor, b: torch.Tensor, before: torch.Tensor) -> torch.Tensor:
    """silu(b + sum_j w[:, j] u_(t - taps + 1 + j)) for rows u [n, channels]; `before` [taps - 1, channels] are the
    rows ahead of them."""
    taps = w.shape[1]
    rows = torch.cat([before, u])
    out = torch.stack([(rows[t:t + taps] * w.T).sum(0) + b for t in range(u.shape[0])])
    return out * torch.sigmoid(out)


def state_space(x: torch.Tensor, B: torch.Tensor, C: torch.Tensor, dt: torch.Tensor, A_log: torch.Tensor, D: torch.Tensor,
                S: torch.Tensor) -> tuple[torch.Tensor, torch.Tensor]:
    """The recurrence, token by token. x [n, H, V], B and C [n, G, N], dt [n, H] (positive), S [H, N, V]:
    S <- exp(-exp(A_log) dt) S + dt B x^T, y = S^T C + D x, head h with group h // (H / G). Returns (y, S)."""
    n, H, _ = x.shape
    G = B.shape[1]
    group = torch.arange(H) // (H // G)
    ys = []
    for t in range(n):
        decay = torch.exp(-torch.exp(A_log) * dt[t])
        S = decay[:, None, None] * S + dt[t][:, None, None] * B[t][group][:, :, None] * x[t][:, None, :]
        ys.append((S * C[t][group][:, :, None]).sum(1) + D[:, None] * x[t])
    return torch.stack(ys), S


def gated_group_norm(y: torch.Tensor, z: torch.Tensor, w: torch.Tensor, parts: int, eps: float) -> torch.Tensor:
    """y silu(z), cut into `parts` equal parts, each divided by its own root mean square; times w."""
    u = y * z * torch.sigmoid(z)
    return unit_rms(u.reshape(u.shape[0], parts, -1), eps).reshape(u.shape) * w


def mamba2(h: torch.Tensor, W: dict, m: dict, eps: float, state: dict) -> torch.Tensor:
    """The "mamba2" mixer; `state` holds S [H, N, V] and the convolution's last inputs."""
    H, V, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    n, inner, taps = h.shape[0], m["heads"] * m["vdim"], W["conv"].shape[1]
    z, u, dt = torch.split(h @ W["in"].T, [inner, inner + 2 * G * N, H], dim=-1)
    if "S" not in state:
        state["S"] = torch.zeros(H, N, V, dtype=h.dtype)
        state["u"] = torch.zeros(taps - 1, u.shape[1], dtype=h.dtype)
    mixed = convolve(u, W["conv"], W["conv.b"], state["u"])
    rows = torch.cat([state["u"], u])
    state["u"] = rows[rows.shape[0] - (taps - 1):]
    x, B, C = torch.split(mixed, [inner, G * N, G * N], dim=-1)
    step = torch.nn.functional.softplus(dt + W["dt_bias"], threshold=1e9)
    y, state["S"] = state_space(x.reshape(n, H, V), B.reshape(n, G, N), C.reshape(n, G, N), step, W["A_log"], W["D"], state["S"])
    return gated_group_norm(y.reshape(n, inner), z, W["norm"], int(m["norm_groups"]), eps) @ W["o"].T


def gated_unit(h: torch.Tensor, W: dict) -> torch.Tensor:
    g = h @ W["gate"].T
    return (g * torch.sigmoid(g) * (h @ W["up"].T)) @ W["down"].T


class PlainMorulix:
    """The whole decoder over one request, fed in any portions; keeps that request's caches and states."""

    def __init__(self, config: dict, weights: dict[str, torch.Tensor], dtype: torch.dtype = torch.float64) -> None:
        self.c, self.dtype = config, dtype
        self.w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
        self.memory: list[dict] = []
        self.fed = 0
        self.after_layers: list[torch.Tensor] = []      # the residual stream after every run of a layer, of the last call

    @classmethod
    def from_folder(cls, folder: str, dtype: torch.dtype = torch.float64) -> "PlainMorulix":
        with open(os.path.join(folder, "config.json")) as f:
            config = json.load(f)
        weights = {}
        with safe_open(os.path.join(folder, "model.safetensors"), "pt", "cpu") as f:
            for name in f.keys():
                weights[name] = f.get_tensor(name)
        return cls(config, weights, dtype)

    def _sub(self, prefix: str) -> dict:
        return {k[len(prefix):]: v for k, v in self.w.items() if k.startswith(prefix)}

    def runs(self) -> list[tuple[int, int | None]]:
        """(layer, number of the pass if the run is a pass's first, else None) in the order of the runs."""
        n, loop = len(self.c["layers"]), self.c.get("loop")
        start, stop, times = (loop["start"], loop["stop"], loop["times"]) if loop else (0, 0, 0)
        out: list[tuple[int, int | None]] = [(i, None) for i in range(start)]
        for t in range(times):
            out += [(i, t if i == start else None) for i in range(start, stop)]
        return out + [(i, None) for i in range(stop, n)]

    def forward(self, tokens: list[int]) -> torch.Tensor:
        """Feeds the request's next tokens; returns logits [len(tokens), vocab]."""
        c, eps = self.c, float(self.c["norm"]["eps"])
        runs = self.runs()
        if not self.memory:
            self.memory = [dict() for _ in runs]
        positions = torch.arange(self.fed, self.fed + len(tokens))
        self.fed += len(tokens)
        x = x0 = self.w["embed"][torch.tensor(tokens)]
        self.after_layers = []
        for memory, (i, t) in zip(self.memory, runs):
            layer = c["layers"][i]
            if t is not None:
                x = pass_input(x, x0, self.w["loop.in"], self.w["loop.step"][t])
            h = layer_norm(x, self.w[f"l{i}.norm1"], eps)
            W, m, kind = self._sub(f"l{i}.mix."), layer["mixer"], layer["type"]
            if kind == "attention":
                add = window_attention(h, positions, W, m, memory)
            elif kind == "latent_attention":
                add = latent_attention(h, positions, W, m, eps, memory)
            elif kind == "mamba2":
                add = mamba2(h, W, m, eps, memory)
            else:
                raise ValueError(kind)
            if layer.get("mlp") is not None:
                add = add + gated_unit(h, self._sub(f"l{i}.mlp."))
            x = x + add
            self.after_layers.append(x.clone())
        return layer_norm(x, self.w["final.norm"], eps) @ self.w["head"].T

    def reset(self) -> None:
        """Forgets the request: the next tokens are a new request's first."""
        self.memory, self.fed = [], 0

    def logits(self, tokens: list[int]) -> torch.Tensor:
        """[len(tokens), vocab] for a request of its own, fed whole."""
        self.reset()
        return self.forward(tokens)

    def streams(self, tokens: list[int]) -> list[torch.Tensor]:
        """The residual stream after every run of a layer, for a request of its own, fed whole."""
        self.logits(tokens)
        return self.after_layers

    def greedy(self, tokens: list[int], n: int) -> list[int]:
        self.reset()
        row, out = self.forward(tokens)[-1], []
        for _ in range(n):
            out.append(int(row.argmax()))
            row = self.forward(out[-1:])[-1]
        return out
