"""A plain, slow implementation of the Derosun decoder: float64, whole sequences at once, one function per
mechanism, nothing shared with the package.  The GPU tests compare the engine with it.

Notation: rows are tokens; ``i`` is a query's position, ``j`` a key's; ``rms(x) = x / sqrt(mean(x^2) + eps)``.

* embedding         ``x = E[token] * scale``
* layer             ``x <- rms(alpha x + mix(x)) w_1``, then ``x <- rms(alpha x + ff(x)) w_2``; the sublayers read the
                    stream itself; a final norm and the head behind the last layer
* latent attention  ``q = W_uq (rms(W_dq h) w_q)``; ``W_dkv h = [c' | r]``, ``c = rms(c') w_c``; ``r`` and every query head's
                    last elements rotated in pairs ``(2e, 2e + 1)`` at YaRN's frequencies, sine and cosine times YaRN's
                    magnitude; head n's key is ``[W_uk,n c | r]``, its value ``W_uv,n c``
* attention         q and k rows normed whole; rotated in pairs ``(e, e + dims/2)`` at frequencies scaled by wavelength;
                    ``softcap tanh(scale q.k / softcap)``; grouped heads
* mlstm             ``S <- exp(f + m - m') S + exp(i - m') k v^T`` and ``n`` likewise with the running maximum
                    ``m' = max(f + m, i)`` from ``m = 0``; ``o = S^T q / (max(|n.q|, exp(-m')) + 1e-6)``; rms per head, a
                    weight per element, a sigmoid gate
* feed-forward      ``W_d (silu(W_g h + b_g) (W_u h + b_u)) + b_d``
"""
import math
from typing import Dict, List, Optional, Sequence

import torch

F = torch.float64


# ---------------------------------------------------------------- configurations
def dense(ff):
    return {"kind": "dense", "ff": ff}


def attention_layer(heads, kv_heads, dim, vdim, rot_dims, base=10000.0, factor=8.0, low=1.0, high=4.0, original=64, scale=None,
                    softcap=15.0, mlp=None):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "softcap": softcap,
                      "scale": scale if scale is not None else 1.5 * dim ** -0.5,
                      "rot": {"base": base, "dims": rot_dims,
                              "scaling": {"factor": factor, "low": low, "high": high, "original": original}}}}


def latent_layer(heads, dim, rot_dim, vdim, q_rank, kv_rank, base=10000.0, factor=4.0, fast=32.0, slow=1.0, original=64, scale=None,
                 mlp=None):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                      "scale": scale if scale is not None else (dim + rot_dim) ** -0.5,
                      "rot": {"base": base, "dims": rot_dim,
                              "scaling": {"factor": factor, "fast": fast, "slow": slow, "original": original}}}}


def mlstm_layer(heads, dim, vdim, gate_cap=9.0, mlp=None):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap}, "mlp": mlp}


def config(layers, vocab=97, width=64, eps=1e-5, alpha=2.0, embed_scale=1.5):
    return {"architecture": "Derosun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "postln_alpha": alpha,
            "embedding": {"scale": embed_scale}, "layers": layers}


def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    e, out = cfg["width"], {}
    out["embed"] = (cfg["vocab"], e)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        out[p + "norm1"] = (e,)
        if layer["mlp"] is not None:
            out[p + "norm2"] = (e,)
        x, H = p + "mix.", m["heads"]
        if layer["type"] == "attention":
            out[x + "q"], out[x + "k"], out[x + "v"] = (H * m["dim"], e), (m["kv_heads"] * m["dim"], e), (m["kv_heads"] * m["vdim"], e)
            out[x + "q.norm"], out[x + "k.norm"] = (H * m["dim"],), (m["kv_heads"] * m["dim"],)
        elif layer["type"] == "latent_attention":
            out[x + "dq"], out[x + "dq.norm"] = (m["q_rank"], e), (m["q_rank"],)
            out[x + "uq"] = (H * (m["dim"] + m["rot_dim"]), m["q_rank"])
            out[x + "dkv"], out[x + "dkv.norm"] = (m["kv_rank"] + m["rot_dim"], e), (m["kv_rank"],)
            out[x + "uk"], out[x + "uv"] = (H * m["dim"], m["kv_rank"]), (H * m["vdim"], m["kv_rank"])
        else:
            out[x + "q"], out[x + "k"] = (H * m["dim"], e), (H * m["dim"], e)
            out[x + "v"], out[x + "g"], out[x + "norm"] = (H * m["vdim"], e), (H * m["vdim"], e), (H * m["vdim"],)
            for gate in ("i", "f"):
                out[x + gate], out[x + gate + ".b"] = (H, e), (H,)
        out[x + "o"] = (e, H * m["vdim"])
        f = layer["mlp"]
        if f is not None:
            for name, shape in (("gate", (f["ff"], e)), ("up", (f["ff"], e)), ("down", (e, f["ff"]))):
                out[p + "mlp." + name], out[p + "mlp." + name + ".b"] = shape, shape[:1]
    out["final.norm"], out["head"] = (e,), (cfg["vocab"], e)
    return out


def random_weights(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """Weights that keep activations of order one, rounded to bfloat16 values (so that a bfloat16 checkpoint holds exactly
    these numbers).  The forget gates lean towards remembering, the input gates spread over both signs.  The matrix memory's
    queries lean towards its keys: a token's read-out is normed to one, so with q and k unrelated the sign of a product q.k
    near zero (all that a first token's read-out has of it) would decide over whole rows, and rounding over the sign."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.rsplit(".", 1)[-1]
        if last in ("norm1", "norm2", "norm"):
            t = 1.0 + 0.1 * torch.randn(shape, generator=g, dtype=F)
        elif name.endswith(".mix.f.b"):
            t = 3.0 + 2.0 * torch.randn(shape, generator=g, dtype=F)
        elif name.endswith(".mix.i.b"):
            t = torch.randn(shape, generator=g, dtype=F)
        elif last == "b":
            t = 0.3 * torch.randn(shape, generator=g, dtype=F)
        elif name == "embed":
            t = torch.randn(shape, generator=g, dtype=F)
        else:
            t = torch.randn(shape, generator=g, dtype=F) / math.sqrt(shape[-1])
        out[name] = t.to(torch.bfloat16).to(F)
    for i, layer in enumerate(cfg["layers"]):
        if layer["type"] == "mlstm":
            p = f"l{i}.mix."
            out[p + "q"] = (0.9 * out[p + "k"] + 0.45 * out[p + "q"]).to(torch.bfloat16).to(F)
    return out


# ---------------------------------------------------------------- mechanisms
def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_of_sum(x, branch, weight, alpha, eps):
    return rms(alpha * x + branch, eps) * weight


def plain_frequencies(rot) -> List[float]:
    return [rot["base"] ** (-2.0 * e / rot["dims"]) for e in range(rot["dims"] // 2)]


def yarn_frequencies(rot) -> List[float]:
    s, d, base = rot["scaling"], rot["dims"], rot["base"]

    def where(turns):
        return d * math.log(s["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(where(s["fast"])), 0), min(math.ceil(where(s["slow"])), d - 1)
    out = []
    for e, f in enumerate(plain_frequencies(rot)):
        r = min(max((e - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / s["factor"] * r + f * (1.0 - r))
    return out


def yarn_magnitude(rot) -> float:
    return 0.1 * math.log(rot["scaling"]["factor"]) + 1.0


def banded_frequencies(rot) -> List[float]:
    """Short wavelengths keep their frequency, long ones are slowed down by the factor, those between are blended."""
    s, out = rot["scaling"], []
    for f in plain_frequencies(rot):
        length = 2 * math.pi / f
        if length < s["original"] / s["high"]:
            out.append(f)
        elif length > s["original"] / s["low"]:
            out.append(f / s["factor"])
        else:
            t = (s["original"] / length - s["low"]) / (s["high"] - s["low"])
            out.append((1 - t) * f / s["factor"] + t * f)
    return out


def turn_halves(x, positions, freq):
    """x [T, heads, n]: its first 2 len(freq) elements in pairs (e, e + len(freq))."""
    n = len(freq)
    a = positions.to(F)[:, None, None] * torch.tensor(freq, dtype=F)
    u, v = x[..., :n], x[..., n:2 * n]
    return torch.cat([u * torch.cos(a) - v * torch.sin(a), v * torch.cos(a) + u * torch.sin(a), x[..., 2 * n:]], -1)


def turn_neighbours(x, positions, freq, magnitude):
    """x [T, heads, n]: its first 2 len(freq) elements in pairs (2e, 2e + 1), sine and cosine times ``magnitude``."""
    n = len(freq)
    a = positions.to(F)[:, None, None] * torch.tensor(freq, dtype=F)
    c, s = torch.cos(a) * magnitude, torch.sin(a) * magnitude
    out = x.clone()
    u, v = x[..., 0:2 * n:2], x[..., 1:2 * n:2]
    out[..., 0:2 * n:2] = u * c - v * s
    out[..., 1:2 * n:2] = v * c + u * s
    return out


def sees(T: int):
    return torch.arange(T)[None, :] <= torch.arange(T)[:, None]


def capped(s, cap):
    return cap * torch.tanh(s / cap)


def softmax_seen(s):
    return torch.softmax(s.masked_fill(~sees(s.shape[-1]), -math.inf), -1)


def attention(h, w, p, m, eps):
    T, H, G, d, vd = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos, freq = torch.arange(T), banded_frequencies(m["rot"])
    q = (rms(h @ w[p + "q"].T, eps) * w[p + "q.norm"]).view(T, H, d)
    k = (rms(h @ w[p + "k"].T, eps) * w[p + "k.norm"]).view(T, G, d)
    q, k, v = turn_halves(q, pos, freq), turn_halves(k, pos, freq), (h @ w[p + "v"].T).view(T, G, vd)
    out = torch.zeros(T, H, vd, dtype=F)
    for n in range(H):
        g = n // (H // G)
        out[:, n] = softmax_seen(capped((q[:, n] @ k[:, g].T) * m["scale"], m["softcap"])) @ v[:, g]
    return out.reshape(T, H * vd) @ w[p + "o"].T


def latent_rows(h, w, p, m, eps):
    """(c [T, kv_rank], r [T, rot_dim]) of every token: what a cache would hold."""
    raw = h @ w[p + "dkv"].T
    c = rms(raw[:, :m["kv_rank"]], eps) * w[p + "dkv.norm"]
    r = turn_neighbours(raw[:, None, m["kv_rank"]:], torch.arange(h.shape[0]), yarn_frequencies(m["rot"]), yarn_magnitude(m["rot"]))
    return c, r[:, 0]


def latent_attention(h, w, p, m, eps):
    T, H, d, rd, vd = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    cq = rms(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]
    q = (cq @ w[p + "uq"].T).view(T, H, d + rd)
    q_plain = q[..., :d]
    q_turned = turn_neighbours(q[..., d:], torch.arange(T), yarn_frequencies(m["rot"]), yarn_magnitude(m["rot"]))
    c, r = latent_rows(h, w, p, m, eps)
    k, v = (c @ w[p + "uk"].T).view(T, H, d), (c @ w[p + "uv"].T).view(T, H, vd)
    out = torch.zeros(T, H, vd, dtype=F)
    for n in range(H):
        out[:, n] = softmax_seen((q_plain[:, n] @ k[:, n].T + q_turned[:, n] @ r.T) * m["scale"]) @ v[:, n]
    return out.reshape(T, H * vd) @ w[p + "o"].T


def log_gates(h, w, p, m):
    """(log input gate, log forget gate) [T, heads]."""
    i = capped(h @ w[p + "i"].T + w[p + "i.b"], m["gate_cap"])
    f = capped(h @ w[p + "f"].T + w[p + "f.b"], m["gate_cap"])
    return i, torch.nn.functional.logsigmoid(f)


def matrix_memory(q, k, v, i, f, state=None):
    """The recurrence of one head over its tokens: q, k [T, d], v [T, vd], log gates [T].  ``state``: (S, n, m) that it goes
    on from; returns (o [T, vd], (S, n, m))."""
    S, n, m = state if state is not None else (torch.zeros(q.shape[1], v.shape[1], dtype=F), torch.zeros(q.shape[1], dtype=F), 0.0)
    out = torch.zeros(q.shape[0], v.shape[1], dtype=F)
    for t in range(q.shape[0]):
        now = max(float(f[t]) + m, float(i[t]))
        keep, write = math.exp(float(f[t]) + m - now), math.exp(float(i[t]) - now)
        S = keep * S + write * torch.outer(k[t], v[t])
        n = keep * n + write * k[t]
        m = now
        out[t] = (S.T @ q[t]) / (max(abs(float(n @ q[t])), math.exp(-m)) + 1e-6)
    return out, (S, n, m)


def mlstm(h, w, p, m, eps):
    T, H, d, vd = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k = (h @ w[p + "q"].T).view(T, H, d) * d ** -0.5, (h @ w[p + "k"].T).view(T, H, d)
    v = (h @ w[p + "v"].T).view(T, H, vd)
    i, f = log_gates(h, w, p, m)
    o = torch.stack([matrix_memory(q[:, n], k[:, n], v[:, n], i[:, n], f[:, n])[0] for n in range(H)], 1)
    y = rms(o, eps).reshape(T, H * vd) * w[p + "norm"] * torch.sigmoid(h @ w[p + "g"].T)
    return y @ w[p + "o"].T


def dense_ff(h, w, p):
    g, u = h @ w[p + "gate"].T + w[p + "gate.b"], h @ w[p + "up"].T + w[p + "up.b"]
    return (g * torch.sigmoid(g) * u) @ w[p + "down"].T + w[p + "down.b"]


MIXERS = {"attention": "attention", "latent_attention": "latent_attention", "mlstm": "mlstm"}


def forward(cfg: dict, weights: Dict[str, torch.Tensor], tokens: Sequence[int], layers_out: Optional[List] = None,
            shake: Optional[torch.Generator] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence.  ``layers_out`` receives the residual stream after every layer.  ``shake``: what a
    sublayer reads and what it returns is multiplied by 1 + 2^-9 noise, as much as rounding to bfloat16 moves it (see
    :func:`sensitivity`)."""
    def s(t):
        return t if shake is None else t * (1.0 + 2.0 ** -9 * torch.randn(t.shape, generator=shake, dtype=F))
    w = {k: v.to(F) for k, v in weights.items()}
    eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
    x = w["embed"][torch.tensor(list(tokens))] * cfg["embedding"]["scale"]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        mix = globals()[MIXERS[layer["type"]]]
        x = norm_of_sum(x, s(mix(s(x), w, p + "mix.", layer["mixer"], eps)), w[p + "norm1"], alpha, eps)
        if layer["mlp"] is not None:
            x = norm_of_sum(x, s(dense_ff(s(x), w, p + "mlp.")), w[p + "norm2"], alpha, eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T


def sensitivity(cfg: dict, weights, tokens: Sequence[int], ref: torch.Tensor, runs: int = 6) -> torch.Tensor:
    """[T]: how far a position's logits move at most when the forward pass is shaken, over some runs.  Most positions move
    little; where a norm divides a read-out that almost cancels, or a latent of one element stands near zero, they move much,
    and no computation in bfloat16 can do better there."""
    g = torch.Generator().manual_seed(len(tokens))
    return torch.stack([(forward(cfg, weights, tokens, shake=g) - ref).abs().max(-1).values for _ in range(runs)]).max(0).values


def argmax_first(row) -> int:
    """The first index of the largest value."""
    return int((row == row.max()).nonzero()[0])
