"""Plain, slow restatement of the Befidra design (torch CPU): one function per mechanism, one sequence at a time, no cache.

TEST INFRASTRUCTURE ONLY: what tests/test_latent_cpu.py and tests/test_gpu_latent.py compare with; the product (triforce_amd/)
never imports it and it imports nothing from the product.  Everything runs in the dtype of the weights it is given (float32 or float64).

``operand`` (everywhere): what happens to an activation right before a matrix product - nothing, or a rounding, which tells how
far a product in a shorter format may move the result.

Notation: T tokens, d = width, H heads, N / R = unrotated / rotated query-key size of a head, V = value size, C = latent size.
"""
import math

import torch


def gelu(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def exact(x):
    return x


def rms(x, eps):
    """x over its root mean square (last dimension)."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def frequencies(rot):
    """Rotation frequencies of the pairs of ``rot`` (dims, base, optional YaRN scaling) and the factor on cos / sin."""
    n, base = rot["dims"], float(rot["base"])
    f = [base ** (-2.0 * i / n) for i in range(n // 2)]
    s = rot.get("scaling")
    if s is None:
        return f, 1.0

    def edge(turns):
        return n * math.log(s["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(edge(s["fast"])), 0)
    hi = min(math.ceil(edge(s["slow"])), n - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / s["factor"] * r + fi * (1.0 - r))
    return out, 0.1 * math.log(s["factor"]) + 1.0


def rotate(x, positions, rot):
    """Interleaved rotation: pair (2i, 2i + 1) of the first rot.dims entries of the last dimension turns by position * f_i.
    x: (T, ..., D)."""
    f, m = frequencies(rot)
    n = rot["dims"]
    a = positions.to(torch.float64)[:, None] * torch.tensor(f, dtype=torch.float64)[None, :]           # (T, n/2)
    shape = (x.shape[0],) + (1,) * (x.dim() - 2) + (n // 2,)
    c, s = (m * torch.cos(a)).to(x.dtype).view(shape), (m * torch.sin(a)).to(x.dtype).view(shape)
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    y = x.clone()
    y[..., 0:n:2] = u * c - v * s
    y[..., 1:n:2] = v * c + u * s
    return y


def latent_attention(h, w, mixer, eps, positions=None, operand=exact):
    """w: the mixer's tensors by short name ("dq", "dq.norm", "uq", "dkv", "dkv.norm", "uk", "uv", "g", "o")."""
    T = h.shape[0]
    H, N, R, V, C = mixer["heads"], mixer["dim"], mixer["rot_dim"], mixer["vdim"], mixer["kv_rank"]
    pos = torch.arange(T) if positions is None else positions
    h = operand(h)
    q = operand(rms(h @ w["dq"].T, eps) * w["dq.norm"]) @ w["uq"].T
    q = q.view(T, H, N + R)
    qn, qr = q[..., :N], rotate(q[..., N:], pos, mixer["rot"])
    kv = h @ w["dkv"].T
    c = operand(rms(kv[:, :C], eps) * w["dkv.norm"])
    kr = rotate(kv[:, C:], pos, mixer["rot"])
    kn = (c @ w["uk"].T).view(T, H, N)
    v = (c @ w["uv"].T).view(T, H, V)
    qn, kn, qr, kr, v = (operand(x) for x in (qn, kn, qr, kr, v))
    s = torch.einsum("thn,shn->hts", qn, kn) + torch.einsum("thr,sr->hts", qr, kr)
    s = s * mixer["scale"]
    s = s.masked_fill(pos[None, None, :] > pos[None, :, None], float("-inf"))
    o = torch.einsum("hts,shv->thv", torch.softmax(s, dim=-1), v).reshape(T, H * V)
    return operand(o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def feed_forward(h, w, operand=exact):
    return operand(gelu(operand(h) @ w["up"].T)) @ w["down"].T


def token_side(x, e, w, eps, operand=exact):
    """Per-layer token input: w has "gate", "proj", "norm"; e is the layer's part of the token's side embedding."""
    y = operand(gelu(operand(x) @ w["gate"].T) * e) @ w["proj"].T
    return rms(y, eps) * w["norm"]


def layer_runs(cfg):
    """(layer, pass, starts a pass) in execution order: layers start .. stop-1 are run ``times`` times in a row."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if loop is None:
        return [(i, 0, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    runs = [(i, 0, False) for i in range(a)]
    for t in range(loop["times"]):
        runs += [(i, t, i == a) for i in range(a, b)]
    return runs + [(i, 0, False) for i in range(b, n)]


def _under(sd, prefix):
    return {k[len(prefix):]: v for k, v in sd.items() if k.startswith(prefix)}


def forward(cfg, sd, tokens, trace=None, operand=exact):
    """tokens: list of ids -> (T, vocab) logits.  ``trace``: list that receives the residual stream after every layer run."""
    ids = torch.as_tensor(tokens, dtype=torch.long)
    eps = cfg["norm"]["eps"]
    x = sd["embed"][ids]
    for i, t, first in layer_runs(cfg):
        L = cfg["layers"][i]
        if first:
            x = x + sd["loop.step"][t]
        h = rms(x, eps) * sd[f"l{i}.norm1"]
        d = latent_attention(h, _under(sd, f"l{i}.mix."), L["mixer"], eps, operand=operand)
        if L.get("mlp") is not None:
            d = d + feed_forward(h, _under(sd, f"l{i}.mlp."), operand)
        x = x + d
        if cfg.get("token_side") is not None:
            n = cfg["token_side"]["dim"]
            x = x + token_side(x, sd["side.embed"][ids][:, i * n:(i + 1) * n], _under(sd, f"l{i}.side."), eps, operand)
        if trace is not None:
            trace.append(x)
    return operand(rms(x, eps) * sd["final.norm"]) @ sd["embed"].T
