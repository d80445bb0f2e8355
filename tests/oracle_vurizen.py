"""A plain, slow float64 statement of the Vurizen decoder, one function per mechanism, written from
the design's equations and sharing no code with the package. ``P`` maps checkpoint tensor names to
float64 tensors, ``cfg`` is the checkpoint's config.json as a dict.

Notation: n tokens, width W. Latent attention: H heads with D unrotated and R rotated query / key
entries and values of size V, all of them read from one latent c (C numbers) and one rotated key
part (R numbers) per token. Gated linear attention: A heads with a D x V state each (rows: key
channel, columns: value channel) that starts at zero.
"""
import math

import torch


def unit_rms(x, eps):
    """x divided by its root mean square over the last axis, eps inside the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, w, b, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w + b


def silu(z):
    return z * torch.sigmoid(z)


# ---- rotation ---------------------------------------------------------------------------------------

def rotary_frequencies(rot):
    """(frequencies [dims / 2], what cos and sin are multiplied by). Plain frequencies
    base^(-2i / dims); with a scaling, entry i runs on a blend of its plain frequency and that
    frequency divided by ``factor``: all plain below the entry whose wavelength makes ``fast`` turns
    in ``original`` positions, all divided above the one that makes ``slow`` turns."""
    dims, base = int(rot["dims"]), float(rot["base"])
    sc = rot.get("scaling")
    out, mag = [], 1.0
    if sc is not None:
        factor = float(sc["factor"])
        mag = 0.1 * math.log(factor) + 1.0

        def entry(turns):
            return dims * math.log(float(sc["original"]) / (2 * math.pi * turns)) / (2 * math.log(base))
        lo = max(math.floor(entry(float(sc["fast"]))), 0)
        hi = min(math.ceil(entry(float(sc["slow"]))), dims - 1)
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if sc is not None:
            ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
            f = f / factor * ramp + f * (1.0 - ramp)
        out.append(f)
    return torch.tensor(out, dtype=torch.float64), mag


def rotate(x, positions, rot):
    """x [n, heads, R] turned on its first ``dims`` entries, entry i with entry i + dims / 2."""
    f, mag = rotary_frequencies(rot)
    half = f.numel()
    ang = positions.double()[:, None, None] * f
    c, s = torch.cos(ang) * mag, torch.sin(ang) * mag
    u, v, rest = x[..., :half], x[..., half:2 * half], x[..., 2 * half:]
    return torch.cat([u * c - v * s, v * c + u * s, rest], -1)


# ---- latent attention -------------------------------------------------------------------------------

def latent_rows(h, P, p, m, eps):
    """What a layer keeps per token: (normed latent [n, C], rotated key part [n, R])."""
    C = int(m["kv_rank"])
    d = h @ P[p + "dkv"].T
    c = unit_rms(d[:, :C], eps) * P[p + "dkv.norm"]
    k_rot = rotate(d[:, None, C:], torch.arange(h.shape[0]), m["rot"])[:, 0]
    return c, k_rot


def visible(n, size):
    """[n, n] mask: position i sees j with 0 <= i - j < size."""
    dist = torch.arange(n)[:, None] - torch.arange(n)[None, :]
    return (dist >= 0) & (dist < size)


def latent_attention(h, P, p, m, kept):
    c, k_rot = kept
    n = h.shape[0]
    H, D, R, V = (int(m[k]) for k in ("heads", "dim", "rot_dim", "vdim"))
    q = (h @ P[p + "q"].T).reshape(n, H, D + R)
    q_rot = rotate(q[:, :, D:], torch.arange(n), m["rot"])
    k = (c @ P[p + "uk"].T).reshape(n, H, D)
    v = (c @ P[p + "uv"].T).reshape(n, H, V)
    see = visible(n, int(m["mask"]["size"]))
    out = []
    for a in range(H):
        score = (q[:, a, :D] @ k[:, a].T + q_rot[:, a] @ k_rot.T) * float(m["scale"])
        out.append(torch.softmax(score.masked_fill(~see, float("-inf")), -1) @ v[:, a])
    return torch.cat(out, -1) @ P[p + "o"].T


# ---- gated linear attention -------------------------------------------------------------------------

def gla_decay(h, P, p, m):
    """Decays [n, A, D] in (0, 1): sigmoid of a low-rank projection plus bias, to the power 1 / tau."""
    z = (h @ P[p + "a1"].T) @ P[p + "a2"].T + P[p + "a2.b"]
    return (torch.sigmoid(z) ** (1.0 / float(m["tau"]))).reshape(h.shape[0], int(m["heads"]), int(m["dim"]))


def gla_scan(q, k, v, alpha):
    """q, k, alpha [n, A, D], v [n, A, V]: the outputs [n, A, V] of
    S_t = diag(alpha_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t from a zero state."""
    n, A, D = q.shape
    S = torch.zeros(A, D, v.shape[-1], dtype=torch.float64)
    out = []
    for t in range(n):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out)


def gla_mixer(h, P, p, m, eps):
    n = h.shape[0]
    A, D, V = (int(m[k]) for k in ("heads", "dim", "vdim"))
    q = (h @ P[p + "q"].T).reshape(n, A, D) * D ** -0.5
    k = (h @ P[p + "k"].T).reshape(n, A, D)
    v = (h @ P[p + "v"].T).reshape(n, A, V)
    o = unit_rms(gla_scan(q, k, v, gla_decay(h, P, p, m)), eps) * P[p + "norm"]
    return (o.reshape(n, A * V) * silu(h @ P[p + "g"].T)) @ P[p + "o"].T


# ---- feed-forward -----------------------------------------------------------------------------------

def gated_expert(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def route(h, router, correction, r):
    """Per token the chosen experts and their weights: lists of ``top`` indices / numbers."""
    E, top = int(r["experts"]), int(r["top"])
    count, keep = int(r["groups"]["count"]), int(r["groups"]["keep"])
    s = torch.sigmoid(h @ router.T)
    chosen, weights = [], []
    for row in s:
        choice = row + correction
        groups = [list(range(g * (E // count), (g + 1) * (E // count))) for g in range(count)]
        value = [sum(sorted((float(choice[e]) for e in g), reverse=True)[:2]) for g in groups]
        kept = sorted(range(count), key=lambda g: -value[g])[:keep]
        allowed = [e for g in kept for e in groups[g]]
        pick = sorted(allowed, key=lambda e: -float(choice[e]))[:top]
        total = sum(float(row[e]) for e in pick) + 1e-20
        chosen.append(pick)
        weights.append([float(row[e]) / total * float(r["scale"]) for e in pick])
    return chosen, weights


def moe_ff(h, P, p, mlp):
    chosen, weights = route(h, P[p + "router"], P[p + "correction"], mlp["router"])
    out = torch.zeros_like(h)
    for t, (pick, wt) in enumerate(zip(chosen, weights)):
        for e, w in zip(pick, wt):
            out[t] += w * gated_expert(h[t:t + 1], P[p + f"e{e}.gate"], P[p + f"e{e}.up"], P[p + f"e{e}.down"])[0]
    return out


# ---- the model --------------------------------------------------------------------------------------

def forward(cfg, P, tokens, keep=None):
    """Logits [n, vocab] of one sequence from position 0; ``keep`` receives the residual stream
    after every layer."""
    eps, mult = float(cfg["norm"]["eps"]), float(cfg["residual_mult"])
    x = P["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    kept = {}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = layer_norm(x, P[p + "norm1"], P[p + "norm1.b"], eps)
        if layer["type"] == "latent_attention":
            src = m.get("kv_from")
            if src is None:
                src = i
                kept[i] = latent_rows(h, P, p + "mix.", m, eps)
            y = latent_attention(h, P, p + "mix.", m, kept[src])
        elif layer["type"] == "gla":
            y = gla_mixer(h, P, p + "mix.", m, eps)
        else:
            raise ValueError(layer["type"])
        x = x + mult * (y * P[p + "ls1"])
        if layer.get("mlp") is not None:
            h = layer_norm(x, P[p + "norm2"], P[p + "norm2.b"], eps)
            x = x + mult * (moe_ff(h, P, p + "mlp.", layer["mlp"]) * P[p + "ls2"])
        if keep is not None:
            keep.append(x.clone())
    return layer_norm(x, P["final.norm"], P["final.norm.b"], eps) @ P["head"].T
