"""A plain, slow implementation of the Kufolorn decoder, one function per mechanism, written from the
design's equations with torch on the CPU (64-bit by default). It shares no code with the engine: it
reads config.json and model.safetensors itself. The tests compare the engine with it.

Notation. rms(x) = x / sqrt(mean(x^2) + eps); n(x) = rms(x) (1 + w) is the layers' norm. Sublayers read the
stream itself and are normed on their way back into it:
    x <- x + n1(mixer(x)),   x <- x + n2(ff(x)).
The mixer is a gated delta rule behind short convolutions ("delta"), or a pair side by side that read the
same input ("parallel"): on the left grouped-query attention over everything before, with biases, norms over
the whole query and key projections, a learned sink and a gate per head; on the right retention, a matrix
state per head with a fixed decay. The feed-forward is a gelu-gated unit, or a mixture of capped experts
scored by a softmax, chosen inside the best groups, the last router outputs standing for experts that hand
their input through. Logits are read with the embedding table and capped by a tanh.
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


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def softcap(z: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(z / cap)


# ---- rotation and attention -------------------------------------------------------------------

def rotate_halves(x: torch.Tensor, positions: torch.Tensor, rot: dict | None) -> torch.Tensor:
    """x [n, heads, D] with rot = {dims, base[, scaling: {factor}]}: the pairs (i, i + dims/2) of every head turn by
    position * base^(-2i/dims) / factor; dimensions from dims on pass."""
    dims = int((rot or {}).get("dims", 0))
    half = dims // 2
    factor = float((rot.get("scaling") or {}).get("factor", 1.0)) if rot else 1.0
    out = x.clone()
    for i in range(half):
        a = positions.to(torch.float64) * (float(rot["base"]) ** (-2.0 * i / dims) / factor)
        c, s = torch.cos(a).to(x.dtype)[:, None], torch.sin(a).to(x.dtype)[:, None]
        u, v = x[:, :, i], x[:, :, i + half]
        out[:, :, i] = u * c - v * s
        out[:, :, i + half] = v * c + u * s
    return out


def sink_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, q_positions: torch.Tensor, scale: float,
                   sinks: torch.Tensor) -> torch.Tensor:
    """q [n, H, D] at `q_positions` over keys k [m, G, D] and values v [m, G, V] at positions 0..m-1, causal;
    weight_j = exp(s_j) / (sum_j' exp(s_j') + exp(sink_h)), s = q.k scale."""
    n, H, _ = q.shape
    G = k.shape[1]
    see = torch.arange(k.shape[0])[None, :] <= q_positions[:, None]
    out = torch.zeros(n, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].T) * scale).masked_fill(~see, float("-inf"))
        top = torch.maximum(s.max(dim=-1, keepdim=True).values, sinks[h])
        e = torch.exp(s - top)
        out[:, h] = (e / (e.sum(-1, keepdim=True) + torch.exp(sinks[h] - top))) @ v[:, g]
    return out


def left_attention(h: torch.Tensor, positions: torch.Tensor, W: dict, m: dict, eps: float, past: dict) -> torch.Tensor:
    """The attention half of the "parallel" mixer for the rows h at `positions`; `past` holds keys and values so far."""
    H, G, D, V = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    n = h.shape[0]
    q = unit_rms(h @ W["q"].T + W["q.b"], eps) * W["q.norm"]                 # over all heads of a token at once
    k = unit_rms(h @ W["k"].T + W["k.b"], eps) * W["k.norm"]
    v = (h @ W["v"].T + W["v.b"]).reshape(n, G, V)
    q = rotate_halves(q.reshape(n, H, D), positions, m.get("rot"))
    k = rotate_halves(k.reshape(n, G, D), positions, m.get("rot"))
    past["k"] = torch.cat([past["k"], k]) if "k" in past else k
    past["v"] = torch.cat([past["v"], v]) if "v" in past else v
    o = sink_attention(q, past["k"], past["v"], positions, float(m["scale"]), W["sink"])
    o = o * torch.sigmoid(h @ W["g"].T)[:, :, None]                          # one gate per head
    return o.reshape(n, H * V) @ W["o"].T


# ---- recurrences ------------------------------------------------------------------------------

def retention_rule(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: torch.Tensor,
                   S: torch.Tensor) -> tuple[torch.Tensor, torch.Tensor]:
    """Token by token: S <- decay_h S + k v^T, o = S^T q. q, k [n, H, D], v [n, H, V], S [H, D, V]. Returns (o, S)."""
    out = []
    for t in range(q.shape[0]):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def retention(h: torch.Tensor, positions: torch.Tensor, W: dict, m: dict, eps: float, state: dict) -> torch.Tensor:
    """The recurrent half of the "parallel" mixer; `state` holds S [H, D, V], zero at the start."""
    H, D, V = (int(m[k]) for k in ("heads", "dim", "vdim"))
    n = h.shape[0]
    q = rotate_halves((h @ W["q"].T).reshape(n, H, D), positions, m.get("rot"))
    k = rotate_halves((h @ W["k"].T).reshape(n, H, D), positions, m.get("rot")) * float(D) ** -0.5
    v = (h @ W["v"].T).reshape(n, H, V)
    if "S" not in state:
        state["S"] = torch.zeros(H, D, V, dtype=h.dtype)
    o, state["S"] = retention_rule(q, k, v, torch.tensor([float(d) for d in m["decay"]], dtype=h.dtype), state["S"])
    return (unit_rms(o, eps).reshape(n, H * V) * silu(h @ W["g"].T)) @ W["o"].T


def convolve(u: torch.Tensor, w: torch.Tensor, before: torch.Tensor) -> torch.Tensor:
    """silu(sum_j w[:, j] u_(t - taps + 1 + j)) for rows u [n, channels]; `before` [taps - 1, channels] are the rows ahead."""
    taps = w.shape[1]
    rows = torch.cat([before, u])
    return silu(torch.stack([(rows[t:t + taps] * w.T).sum(0) for t in range(u.shape[0])]))


def unit_vectors(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, g: torch.Tensor, beta: torch.Tensor,
               S: torch.Tensor) -> tuple[torch.Tensor, torch.Tensor]:
    """Token by token: S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q. q, k [n, H, D], v [n, H, V],
    g, beta [n, H], S [H, D, V]. Returns (o, S)."""
    out = []
    for t in range(q.shape[0]):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def delta_mixer(h: torch.Tensor, W: dict, m: dict, eps: float, state: dict) -> torch.Tensor:
    """The "delta" mixer; `state` holds S [H, D, V] and the last taps - 1 projected rows of q, k and v."""
    H, G, D, V = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    n = h.shape[0]
    mixed = {}
    for name in ("q", "k", "v"):
        u, w = h @ W[name].T, W[f"{name}.conv"]
        before = state.get(name, torch.zeros(w.shape[1] - 1, u.shape[1], dtype=h.dtype))
        mixed[name] = convolve(u, w, before)
        rows = torch.cat([before, u])
        state[name] = rows[rows.shape[0] - (w.shape[1] - 1):]
    own = torch.arange(H) // (H // G)                                        # a head's q/k head
    q = unit_vectors(mixed["q"].reshape(n, G, D))[:, own] * float(D) ** -0.5
    k = unit_vectors(mixed["k"].reshape(n, G, D))[:, own]
    beta = torch.sigmoid(h @ W["b"].T)
    step = torch.nn.functional.softplus(h @ W["a"].T + W["dt_bias"], threshold=1e9)
    g = torch.exp(-torch.exp(W["A_log"]) * step)
    if "S" not in state:
        state["S"] = torch.zeros(H, D, V, dtype=h.dtype)
    o, state["S"] = delta_rule(q, k, mixed["v"].reshape(n, H, V), g, beta, state["S"])
    o = unit_rms(o, eps) * W["norm"] * silu(h @ W["g"].T).reshape(n, H, V)
    return o.reshape(n, H * V) @ W["o"].T


# ---- feed-forwards ----------------------------------------------------------------------------

def dense_unit(h: torch.Tensor, W: dict) -> torch.Tensor:
    return (gelu_tanh(h @ W["gate"].T) * (h @ W["up"].T)) @ W["down"].T


def capped_expert(h: torch.Tensor, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor, limit: float) -> torch.Tensor:
    g, u = torch.clamp(h @ gate.T, max=limit), torch.clamp(h @ up.T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ down.T


def choose(z: torch.Tensor, correction: torch.Tensor, top: int, groups: int, keep: int) -> tuple[list[int], list[float]]:
    """The experts chosen for one token with router logits z, and their weights: scores s = softmax(z); among the
    experts of the `keep` groups (equal stretches of neighbours) with the largest best s + correction, the `top` with the
    largest s + correction; the weights are their s."""
    s = torch.softmax(z, dim=-1)
    choice = s + correction
    size = z.shape[0] // groups
    best = sorted(range(groups), key=lambda a: -float(choice[a * size:(a + 1) * size].max()))[:keep]
    allowed = [e for e in range(z.shape[0]) if e // size in best]
    chosen = sorted(allowed, key=lambda e: -float(choice[e]))[:top]
    return chosen, [float(s[e]) for e in chosen]


def choice_margin(z: torch.Tensor, correction: torch.Tensor, top: int, groups: int, keep: int) -> float:
    """By how much of its score (the larger of the two scores) the weakest thing chosen is ahead of the strongest one left
    out, expert or group, whichever is closer: a small number is a choice that rounding may turn round."""
    s = torch.softmax(z, dim=-1)
    choice = s + correction
    size = z.shape[0] // groups
    lead = [max(range(a * size, (a + 1) * size), key=lambda e: float(choice[e])) for a in range(groups)]
    lead.sort(key=lambda e: -float(choice[e]))
    allowed = sorted((e for a in lead[:keep] for e in range(a // size * size, (a // size + 1) * size)), key=lambda e: -float(choice[e]))
    pairs = ([(lead[keep - 1], lead[keep])] if keep < groups else []) + ([(allowed[top - 1], allowed[top])] if top < len(allowed) else [])
    return min((float(choice[a] - choice[b]) / float(max(s[a], s[b])) for a, b in pairs), default=math.inf)


def experts_unit(h: torch.Tensor, W: dict, c: dict) -> torch.Tensor:
    router = c["router"]
    real, groups = int(router["experts"]), router.get("groups") or {"count": 1, "keep": 1}
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        chosen, weights = choose(W["router"] @ h[t], W["correction"], int(router["top"]), int(groups["count"]), int(groups["keep"]))
        for e, s in zip(chosen, weights):
            y = capped_expert(h[t], W[f"e{e}.gate"], W[f"e{e}.up"], W[f"e{e}.down"], float(c["expert"]["limit"])) if e < real else h[t]
            out[t] += s * y
    return out


class PlainKufolorn:
    """The whole decoder over one request, fed in any portions; keeps that request's caches and states."""

    def __init__(self, config: dict, weights: dict[str, torch.Tensor], dtype: torch.dtype = torch.float64) -> None:
        self.c, self.dtype = config, dtype
        self.w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
        self.memory: list[dict] = []
        self.fed = 0
        self.after_layers: list[torch.Tensor] = []      # the residual stream after every layer, of the last call
        self.margin = math.inf                          # the closest call of any router, of the last call (`choice_margin`)

    @classmethod
    def from_folder(cls, folder: str, dtype: torch.dtype = torch.float64) -> "PlainKufolorn":
        with open(os.path.join(folder, "config.json")) as f:
            config = json.load(f)
        weights = {}
        with safe_open(os.path.join(folder, "model.safetensors"), "pt", "cpu") as f:
            for name in f.keys():
                weights[name] = f.get_tensor(name)
        return cls(config, weights, dtype)

    def _sub(self, prefix: str) -> dict:
        return {k[len(prefix):]: v for k, v in self.w.items() if k.startswith(prefix)}

    def mixer(self, i: int, x: torch.Tensor, positions: torch.Tensor, memory: dict) -> torch.Tensor:
        layer, eps = self.c["layers"][i], float(self.c["norm"]["eps"])
        m, kind = layer["mixer"], layer["type"]
        if kind == "delta":
            return delta_mixer(x, self._sub(f"l{i}.mix."), m, eps, memory)
        if kind != "parallel":
            raise ValueError(kind)
        left = left_attention(x, positions, self._sub(f"l{i}.mix.left."), m["left"], eps, memory)
        right = retention(x, positions, self._sub(f"l{i}.mix.right."), m["right"], eps, memory)
        return float(m["left_scale"]) * left + float(m["right_scale"]) * right

    def forward(self, tokens: list[int]) -> torch.Tensor:
        """Feeds the request's next tokens; returns logits [len(tokens), vocab]."""
        c, eps = self.c, float(self.c["norm"]["eps"])
        if not self.memory:
            self.memory = [dict() for _ in c["layers"]]
        positions = torch.arange(self.fed, self.fed + len(tokens))
        self.fed += len(tokens)
        x = self.w["embed"][torch.tensor(tokens)]
        self.after_layers, self.margin = [], math.inf
        for i, layer in enumerate(c["layers"]):
            x = x + layer_norm(self.mixer(i, x, positions, self.memory[i]), self.w[f"l{i}.norm1"], eps)
            mlp = layer.get("mlp")
            if mlp is not None:
                W = self._sub(f"l{i}.mlp.")
                if mlp["kind"] == "moe":
                    r = mlp["router"]
                    g = r.get("groups") or {"count": 1, "keep": 1}
                    self.margin = min([self.margin] + [choice_margin(W["router"] @ h, W["correction"], r["top"], g["count"], g["keep"]) for h in x])
                y = dense_unit(x, W) if mlp["kind"] == "dense" else experts_unit(x, W, mlp)
                x = x + layer_norm(y, self.w[f"l{i}.norm2"], eps)
            self.after_layers.append(x.clone())
        logits = layer_norm(x, self.w["final.norm"], eps) @ self.w["embed"].T
        cap = float(c.get("logit_softcap") or 0.0)
        return softcap(logits, cap) if cap else logits

    def reset(self) -> None:
        """Forgets the request: the next tokens are a new request's first."""
        self.memory, self.fed = [], 0

    def logits(self, tokens: list[int]) -> torch.Tensor:
        """[len(tokens), vocab] for a request of its own, fed whole."""
        self.reset()
        return self.forward(tokens)

    def streams(self, tokens: list[int]) -> list[torch.Tensor]:
        """The residual stream after every layer, for a request of its own, fed whole."""
        self.logits(tokens)
        return self.after_layers

    def greedy(self, tokens: list[int], n: int) -> list[int]:
        self.reset()
        row, out = self.forward(tokens)[-1], []
        for _ in range(n):
            out.append(int(row.argmax()))
            row = self.forward(out[-1:])[-1]
        return out
