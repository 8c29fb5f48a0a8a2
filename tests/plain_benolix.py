"""A plain, slow implementation of the Benolix design, one function per mechanism, in float64.  It shares no code
with the engine: the CPU and GPU tests compare the engine with it.

Notation: T tokens, W the model's width, H heads.  Linear weights are [out, in].  A sequence is processed in any
number of calls of ``PlainBenolix.forward``; between calls the model keeps, for every layer that projects keys of its
own, the latents and rotated key parts of all tokens (nothing is ever dropped: what a query may see is the mask's
business alone).
"""

from __future__ import annotations

import math

import torch

F = torch.float64


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def silu(z):
    return z / (1 + torch.exp(-z))


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


# ----------------------------------------------------------------------------- positions and masks


def rotate_neighbours(x, positions, dims: int, base: float):
    """x [T, ..., n]: entries 2i and 2i + 1 of the first ``dims`` turn together by ``position * base^(-2i/dims)``."""
    out = x.clone()
    for i in range(dims // 2):
        a = positions.to(F) * base ** (-2.0 * i / dims)
        c, s = torch.cos(a), torch.sin(a)
        while c.dim() < x.dim() - 1:
            c, s = c.unsqueeze(-1), s.unsqueeze(-1)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def window_mask(query_positions, key_positions, size: int | None):
    """[T, n] booleans: a query sees itself and the ``size - 1`` tokens before it (None: all before it)."""
    back = query_positions[:, None] - key_positions[None, :]
    seen = back >= 0
    if size is not None:
        seen = seen & (back < size)
    return seen


# ----------------------------------------------------------------------------- attention over latents


def query_from_latent(h, w, m, eps):
    """[T, H, dim + rot_dim]: h is projected down, normed, and projected up head by head."""
    c = rms(h @ w["dq"].T, eps) * w["dq.norm"]
    return (c @ w["uq"].T).view(h.shape[0], m["heads"], m["dim"] + m["rot_dim"])


def key_rows(h, positions, w, m, eps):
    """What a layer leaves for each token: (latent [T, rank], rotated key part [T, rot_dim])."""
    rank, rot = m["kv_rank"], m["rot"]
    down = h @ w["dkv"].T
    return (rms(down[:, :rank], eps) * w["dkv.norm"],
            rotate_neighbours(down[:, rank:], positions, rot["dims"], rot["base"]))


def attend(q, positions, latents, rotated, w, m):
    """q [T, H, dim + rot_dim] with its rotated part turned; keys and values expanded from the latents.  Returns
    [T, H, vdim]."""
    H, d = m["heads"], m["dim"]
    n = latents.shape[0]
    k = (latents @ w["uk"].T).view(n, H, d)
    v = (latents @ w["uv"].T).view(n, H, m["vdim"])
    scores = torch.einsum("thd,nhd->htn", q[..., :d], k) + torch.einsum("thr,nr->htn", q[..., d:], rotated)
    seen = window_mask(positions, torch.arange(n), (m.get("mask") or {}).get("size"))
    scores = (scores * m["scale"]).masked_fill(~seen[None], -math.inf)
    e = torch.exp(scores - scores.max(dim=-1, keepdim=True).values)
    return torch.einsum("htn,nhv->thv", e / e.sum(dim=-1, keepdim=True), v)


def gate_entries(o, h, w):
    """Every entry of the concatenated heads times the sigmoid of a projection of h."""
    return o * sigmoid(h @ w["g"].T)


def latent_mixer(h, positions, w, m, eps, rows):
    """``rows``: (latents, rotated key parts) of all tokens so far, this call's included."""
    q = query_from_latent(h, w, m, eps)
    d, rot = m["dim"], m["rot"]
    q = torch.cat((q[..., :d], rotate_neighbours(q[..., d:], positions, rot["dims"], rot["base"])), dim=-1)
    o = attend(q, positions, rows[0], rows[1], w, m).reshape(h.shape[0], -1)
    return gate_entries(o, h, w) @ w["o"].T


# ----------------------------------------------------------------------------- feed-forwards


def dense_ff(h, w):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def clamped_gate(g, u, limit: float):
    """min(g, limit) * sigmoid(1.702 min(g, limit)) * (clamp(u) + 1)."""
    g = torch.minimum(g, torch.tensor(limit, dtype=g.dtype))
    return g * sigmoid(1.702 * g) * (torch.clamp(u, -limit, limit) + 1)


def router_scores(h, w):
    z = h @ w["router"].T
    e = torch.exp(z - z.max(dim=-1, keepdim=True).values)
    return e / e.sum(dim=-1, keepdim=True)


def routed_choice(scores, correction, top: int, scale: float):
    """(chosen outputs [T, top], their weights [T, top]): the correction matters to the choice alone."""
    chosen = torch.topk(scores + correction, top, dim=-1).indices
    s = torch.gather(scores, 1, chosen)
    return chosen, s / (s.sum(dim=-1, keepdim=True) + 1e-20) * scale


def routed_margin(scores, correction, top: int):
    """Per token, how far the last chosen output's choice score lies above the best one left out."""
    pick = scores + correction
    if top >= pick.shape[-1]:
        return torch.full((pick.shape[0],), math.inf, dtype=pick.dtype)
    best = torch.topk(pick, top + 1, dim=-1).values
    return best[:, top - 1] - best[:, top]


def routed_ff(h, w, mlp, margins=None):
    r, limit = mlp["router"], mlp["expert"]["limit"]
    scores = router_scores(h, w)
    if margins is not None:
        margins.append(routed_margin(scores, w["correction"], r["top"]))
    chosen, weights = routed_choice(scores, w["correction"], r["top"], r.get("scale", 1.0))
    out = torch.zeros_like(h)
    for e in range(r["experts"] + r.get("identity", 0)):
        share = (weights * (chosen == e)).sum(dim=-1, keepdim=True)
        if e < r["experts"]:
            y = clamped_gate(h @ w[f"e{e}.gate"].T, h @ w[f"e{e}.up"].T, limit) @ w[f"e{e}.down"].T
        else:
            y = h
        out = out + share * y
    return out


# ----------------------------------------------------------------------------- the model


def under(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


class PlainBenolix:
    def __init__(self, cfg: dict, tensors: dict):
        self.cfg = cfg
        self.t = {k: (v.to(F) if v.is_floating_point() else v) for k, v in tensors.items()}
        self.seen = 0
        self.rows: dict[int, tuple] = {}     # layer -> (latents, rotated key parts)

    def norm(self, x, name):
        return rms(x, self.cfg["norm"]["eps"]) * (1 + self.t[name])

    def forward(self, ids, trail=None, margins=None):
        """Logits [len(ids), vocab] of the sequence's next tokens.  ``trail`` receives the stream after every layer,
        ``margins`` every routed layer's ``routed_margin``."""
        cfg, T = self.cfg, len(ids)
        eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
        positions = torch.arange(self.seen, self.seen + T)
        x = self.t["embed"][torch.tensor(ids)] * cfg["embedding"]["scale"]
        for i, layer in enumerate(cfg["layers"]):
            p, m = f"l{i}.", layer["mixer"]
            w = under(self.t, p + "mix.")
            source = m.get("kv_from")
            if source is None:
                new = key_rows(x, positions, w, m, eps)
                old = self.rows.get(i)
                self.rows[i] = new if old is None else tuple(torch.cat((a, b)) for a, b in zip(old, new))
                source = i
            x = self.norm(alpha * x + latent_mixer(x, positions, w, m, eps, self.rows[source]), p + "norm1")
            mlp = layer.get("mlp")
            if mlp is not None:
                w = under(self.t, p + "mlp.")
                y = dense_ff(x, w) if mlp["kind"] == "dense" else routed_ff(x, w, mlp, margins)
                x = self.norm(alpha * x + y, p + "norm2")
            elif p + "norm2" in self.t:
                x = self.norm(alpha * x, p + "norm2")
            if trail is not None:
                trail.append(x)
        self.seen += T
        return self.norm(x, "final.norm") @ self.t["head"].T
