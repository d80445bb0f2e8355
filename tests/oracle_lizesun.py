"""A plain, slow float64 statement of the Lizesun decoder, one function per mechanism, written from
the design's equations and sharing no code with the package. ``P`` maps checkpoint tensor names to
float64 tensors, ``cfg`` is the checkpoint's config.json as a dict.

Notation: n tokens, width W; attention with H query heads over G key / value heads (query head a
reads key / value head a // (H / G)), key size D, value size E; recurrences keep a D x E state per
head (rows: key channel, columns: value channel) that starts at zero.
"""
import torch


# ---- norms ------------------------------------------------------------------------------------------

def tanh_norm(x, alpha, w, b):
    """Dynamic Tanh: no mean, no variance."""
    return torch.tanh(alpha * x) * w + b


def unit_rms(x, eps):
    """x divided by its root mean square over the last axis, eps inside the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit_length(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def silu(z):
    return z * torch.sigmoid(z)


def model_norm(x, P, name):
    return tanh_norm(x, P[name + ".alpha"], P[name], P[name + ".b"])


# ---- attention --------------------------------------------------------------------------------------

def turn_halves(x, pos, base, dims):
    """x [n, heads, D]: entry i pairs with entry i + dims / 2 on the leading ``dims`` entries; pair i
    of the token at position p turns by p * base^(-2 i / dims)."""
    r = dims // 2
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(r)], dtype=torch.float64)
    ang = pos.to(torch.float64)[:, None, None] * f
    c, s = torch.cos(ang), torch.sin(ang)
    u, v = x[..., :r], x[..., r:dims]
    out = x.clone()
    out[..., :r] = u * c - v * s
    out[..., r:dims] = v * c + u * s
    return out


def seen_chunk(n, size):
    """[i, j]: j <= i in the same chunk of ``size`` positions, counted from position 0."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None]
    return (j <= i) & (i // size == j // size)


def seen_window(n, size, keep_first):
    """[i, j]: j <= i, and j less than ``size`` back or among the first ``keep_first``."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None]
    return (j <= i) & ((i - j < size) | (j < keep_first))


def attend(q, k, v, seen, scale, softcap=None, sink=None):
    """q [n, H, D], k [n, G, D], v [n, G, E], seen [n, n]. ``softcap`` c: the scaled score becomes
    c tanh(score / c). ``sink`` [H]: exp(sink) joins the softmax denominator."""
    n, H, _ = q.shape
    G, E = v.shape[1], v.shape[2]
    out = torch.zeros(n, H, E, dtype=torch.float64)
    for a in range(H):
        g = a // (H // G)
        s = (q[:, a] @ k[:, g].T) * scale
        if softcap is not None:
            s = softcap * torch.tanh(s / softcap)
        s = s.masked_fill(~seen, float("-inf"))
        if sink is not None:
            s = torch.cat([s, sink[a].expand(n, 1)], 1)
        p = torch.softmax(s, -1)
        out[:, a] = p[:, :n] @ v[:, g]
    return out


def chunked_attention(h, P, p, m, eps, v_first=None):
    """The mixer 'attention'; returns (output, this layer's mixed values). ``v_first`` [n, G, E]: the
    first value-mixing layer's values (None: this layer takes its own as they are)."""
    n = h.shape[0]
    H, G, D, E = (int(m[x]) for x in ("heads", "kv_heads", "dim", "vdim"))
    q = (h @ P[p + "q"].T + P[p + "q.b"]).reshape(n, H, D)
    k = (h @ P[p + "k"].T + P[p + "k.b"]).reshape(n, G, D)
    v = (h @ P[p + "v"].T + P[p + "v.b"]).reshape(n, G, E)
    q, k = unit_rms(q, eps) * P[p + "q.norm"], unit_rms(k, eps) * P[p + "k.norm"]
    if v_first is not None:
        lam = P[p + "vmix"]
        v = (1 - lam) * v + lam * v_first
    seen = seen_chunk(n, int(m["mask"]["size"])) if m.get("mask") else torch.ones(n, n).tril().bool()
    o = attend(q, k, v, seen, float(m["scale"]), m.get("softcap"))
    o = o * torch.sigmoid(h @ P[p + "g"].T)[:, :, None]
    return o.reshape(n, H * E) @ P[p + "o"].T, v


def window_attention(h, P, p, m, eps):
    """The left half of the mixer 'parallel'."""
    n = h.shape[0]
    H, G, D, E = (int(m[x]) for x in ("heads", "kv_heads", "dim", "vdim"))
    pos = torch.arange(n)
    q, k = (h @ P[p + "q"].T).reshape(n, H, D), (h @ P[p + "k"].T).reshape(n, G, D)
    v = (h @ P[p + "v"].T).reshape(n, G, E)
    if m.get("rot"):
        base, dims = float(m["rot"]["base"]), int(m["rot"]["dims"])
        q, k = turn_halves(q, pos, base, dims), turn_halves(k, pos, base, dims)
    q, k = unit_rms(q, eps), unit_rms(k, eps)
    mask = m.get("mask")
    seen = seen_window(n, int(mask["size"]), int(mask.get("keep_first", 0))) if mask else torch.ones(n, n).tril().bool()
    o = attend(q, k, v, seen, float(m["scale"]), None, P[p + "sink"])
    return o.reshape(n, H * E) @ P[p + "o"].T


# ---- recurrences ------------------------------------------------------------------------------------

def causal_conv(h, w):
    """h [n, C], w [C, taps]: a causal convolution over time per channel, the last tap on the current
    token, zeros ahead of the sequence."""
    taps = w.shape[1]
    out = torch.zeros_like(h)
    for j in range(taps):
        back = taps - 1 - j
        if back < h.shape[0]:
            out[back:] += h[:h.shape[0] - back] * w[:, j]
    return out


def corrected_sum(q, k, v, beta, g):
    """One head; q, k, g [n, D], v [n, E], beta [n]: S <- diag(g_t) S; u = beta_t (v_t - S^T k_t);
    S <- S + k_t u^T; o_t = S^T q_t."""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=torch.float64)
    out = []
    for t in range(q.shape[0]):
        S = g[t][:, None] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + torch.outer(k[t], u)
        out.append(S.T @ q[t])
    return torch.stack(out)


def channel_decay(h, P, p, A, D):
    """[n, A, D]: exp(-exp(A_log) softplus(low-rank path + dt_bias)) per head and key channel."""
    z = (h @ P[p + "a1"].T) @ P[p + "a2"].T + P[p + "dt_bias"]
    sp = torch.logaddexp(z, torch.zeros_like(z)).reshape(-1, A, D)
    return torch.exp(-torch.exp(P[p + "A_log"])[None, :, None] * sp)


def channel_delta(h, P, p, m, eps):
    """The mixer 'channel_delta'."""
    n = h.shape[0]
    A, G, D, E = (int(m[x]) for x in ("heads", "kv_heads", "dim", "vdim"))
    q = silu(causal_conv(h @ P[p + "q"].T, P[p + "q.conv"])).reshape(n, G, D)
    k = silu(causal_conv(h @ P[p + "k"].T, P[p + "k.conv"])).reshape(n, G, D)
    v = silu(causal_conv(h @ P[p + "v"].T, P[p + "v.conv"])).reshape(n, A, E)
    q, k = unit_length(q) * D ** -0.5, unit_length(k)
    beta = torch.sigmoid(h @ P[p + "b"].T)
    g = channel_decay(h, P, p, A, D)
    o = torch.stack([corrected_sum(q[:, i // (A // G)], k[:, i // (A // G)], v[:, i], beta[:, i], g[:, i])
                     for i in range(A)], 1)
    o = (unit_rms(o, eps) * P[p + "norm"]).reshape(n, A * E)
    return (o * torch.sigmoid((h @ P[p + "g1"].T) @ P[p + "g2"].T)) @ P[p + "o"].T


def matrix_memory(q, k, v, i, f):
    """One head; q, k [n, D], v [n, E], i, f [n] the log input and log forget gates. Exponential gates
    under a running maximum that starts at 0."""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=torch.float64)
    N = torch.zeros(k.shape[1], dtype=torch.float64)
    m = torch.zeros((), dtype=torch.float64)
    out = []
    for t in range(q.shape[0]):
        new = torch.maximum(f[t] + m, i[t])
        keep, write = torch.exp(f[t] + m - new), torch.exp(i[t] - new)
        S = keep * S + write * torch.outer(k[t], v[t])
        N = keep * N + write * k[t]
        m = new
        out.append(S.T @ q[t] / (torch.maximum((N @ q[t]).abs(), torch.exp(-m)) + 1e-6))
    return torch.stack(out)


def memory_gates(h, P, p, cap):
    """(log input gate, log forget gate) [n, heads] of the matrix memory."""
    i = cap * torch.tanh((h @ P[p + "i"].T + P[p + "i.b"]) / cap)
    f = cap * torch.tanh((h @ P[p + "f"].T + P[p + "f.b"]) / cap)
    return i, -torch.logaddexp(-f, torch.zeros_like(f))


def memory_mixer(h, P, p, m, eps):
    """The right half of the mixer 'parallel'."""
    n = h.shape[0]
    A, D, E = (int(m[x]) for x in ("heads", "dim", "vdim"))
    q = (h @ P[p + "q"].T).reshape(n, A, D) * D ** -0.5
    k = (h @ P[p + "k"].T).reshape(n, A, D)
    v = (h @ P[p + "v"].T).reshape(n, A, E)
    i, f = memory_gates(h, P, p, float(m["gate_cap"]))
    o = torch.stack([matrix_memory(q[:, a], k[:, a], v[:, a], i[:, a], f[:, a]) for a in range(A)], 1)
    o = unit_rms(o, eps).reshape(n, A * E) * P[p + "norm"]
    return (o * torch.sigmoid(h @ P[p + "g"].T)) @ P[p + "o"].T


# ---- the model --------------------------------------------------------------------------------------

def squared_relu_ff(h, up, down):
    return torch.relu(h @ up.T) ** 2 @ down.T


def forward(cfg, P, tokens, keep=None):
    """Logits [n, vocab] of one sequence from position 0; ``keep`` receives the residual stream
    after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = P["embed"][torch.as_tensor(tokens, dtype=torch.long)] * float(cfg["embedding"]["scale"])
    v_first = None
    for l, layer in enumerate(cfg["layers"]):
        p, m = f"l{l}.", layer["mixer"]
        h = model_norm(x, P, p + "norm1")
        if layer["type"] == "channel_delta":
            y = channel_delta(h, P, p + "mix.", m, eps)
        elif layer["type"] == "attention":
            mixing = bool(m.get("v_mix"))
            y, v = chunked_attention(h, P, p + "mix.", m, eps, v_first if mixing else None)
            if mixing and v_first is None:
                v_first = v
        elif layer["type"] == "parallel":
            y = (float(m["left_scale"]) * window_attention(h, P, p + "mix.left.", m["left"], eps) +
                 float(m["right_scale"]) * memory_mixer(h, P, p + "mix.right.", m["right"], eps))
        else:
            raise ValueError(layer["type"])
        x = x + y
        if layer.get("mlp") is not None:
            x = x + squared_relu_ff(model_norm(x, P, p + "norm2"), P[p + "mlp.up"], P[p + "mlp.down"])
        if keep is not None:
            keep.append(x.clone())
    return model_norm(x, P, "final.norm") @ P["head"].T
