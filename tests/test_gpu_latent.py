"""Befidra on the device: every kernel against plain torch fp32 / fp64, every mechanism and schedule against oracle/ref_latent.py,
in float32 (sharp) and bfloat16."""
import json

import pytest
import torch

from oracle import ref_latent as R
from tests import latent_helpers as H

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]
F32 = 5e-5                                                    # H.bound in float32
OP = {torch.float32: dict(atol=3e-5, rtol=3e-5), torch.bfloat16: dict(atol=2e-2, rtol=2e-2)}
DEV = "cuda:0"


@pytest.fixture(scope="module")
def ol():
    from triforce_amd import ops_latent
    return ops_latent


def rnd(*shape, seed=0, dtype=torch.float32, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * scale).to(dtype).to(DEV)


class Geom:
    def __init__(self, H, N, R, V, C, Q, c_real=None, q_real=None):
        self.H, self.N, self.R, self.V, self.C, self.Q = H, N, R, V, C, Q
        self.c_real, self.q_real = c_real or C, q_real or Q


class Rope:
    def __init__(self, n, half):
        a = torch.rand(n, half, generator=torch.Generator().manual_seed(1)) * 6.28
        self.cos, self.sin, self.half, self.max_pos = (1.1 * a.cos()).to(DEV), (1.1 * a.sin()).to(DEV), half, n

    def turn(self, x, pos):
        """x (rows, ..., R)"""
        c, s = self.cos[pos.long()], self.sin[pos.long()]
        c, s = (t.view(t.shape[0], *[1] * (x.dim() - 2), self.half) for t in (c, s))
        y = x.clone()
        u, v = x[..., 0:2 * self.half:2], x[..., 1:2 * self.half:2]
        y[..., 0:2 * self.half:2], y[..., 1:2 * self.half:2] = u * c - v * s, v * c + u * s
        return y


def f(t):
    return t.float()


# ---- skinny GEMM and its epilogues ------------------------------------------------------------------------------------------
ROWS = [1, 3, 16, 17, 33, 70]


def octets(x):
    rows, k = x.shape
    return x.view(rows, k // 8, 8).permute(1, 0, 2).contiguous()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", ROWS)
@pytest.mark.parametrize("n,k,n_real", [(32, 32, 17), (96, 416, 96), (2080, 96, 2077), (5024, 1056, 5001), (10272, 64, 10272), (13472, 160, 13469)])
def test_linear_f32(ol, dtype, rows, n, k, n_real):
    w, x = rnd(n, k, seed=1, dtype=dtype), rnd(rows, k, seed=2, dtype=dtype)
    wt = ol.TileWeight(w)
    y = ol.linear_f32(x, wt, n_real)
    assert torch.equal(ol.act_rows(octets(x)), x) and torch.equal(ol.linear_f32(octets(x), wt, n_real), y)
    torch.testing.assert_close(y, (f(x) @ f(w).T)[:, :n_real], atol=2e-4 * k ** 0.5, rtol=1e-4)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", ROWS)
@pytest.mark.parametrize("n_raw,n_up", [(224, 0), (224, 96), (224, 13312)])
def test_input_projection(ol, dtype, rows, n_raw, n_up):
    k, off = 160, 64
    w, x = rnd(n_raw + n_up, k, seed=1, dtype=dtype, scale=k ** -0.5), rnd(rows, k, seed=2, dtype=dtype)
    act = torch.full((rows, off + n_up), 7.0, dtype=dtype, device=DEV)
    qw = rnd(96, seed=9)
    raw, ss, xq = ol.input_projection(x, ol.TileWeight(w), n_raw, qw, act, off)
    want = f(x) @ f(w).T
    torch.testing.assert_close(raw, want[:, :n_raw], atol=1e-4, rtol=1e-4)
    torch.testing.assert_close(f(ol.act_rows(xq)), want[:, :96] * qw, **OP[dtype])
    torch.testing.assert_close(ss, want[:, :n_raw].view(rows, -1, 16).pow(2).sum(-1), atol=1e-3, rtol=1e-3)
    torch.testing.assert_close(f(act[:, off:]), R.gelu(want[:, n_raw:]), **OP[dtype])
    assert bool((act[:, :off] == 7).all())
    block = torch.full(((off + n_up) // 8, rows, 8), 7.0, dtype=dtype, device=DEV)
    raw2, ss2, xq2 = ol.input_projection(octets(x), ol.TileWeight(w), n_raw, qw, block, off)
    assert torch.equal(ol.act_rows(block), act) and torch.equal(xq2, xq) and torch.equal(raw2, raw) and torch.equal(ss2, ss)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", ROWS)
@pytest.mark.parametrize("g", [Geom(3, 32, 32, 32, 64, 96, c_real=50, q_real=70), Geom(1, 64, 32, 32, 32, 32, c_real=9, q_real=7)])
def test_query_and_append(ol, dtype, rows, g):
    eps, half = 1e-3, g.R // 2 - 3                                # the last pairs are not rotated
    rope = Rope(300, half)
    width = g.Q + g.C + g.R + 64
    raw = rnd(rows, width, seed=3)
    raw[:, g.q_real:g.Q] = 0
    raw[:, g.Q + g.c_real:g.Q + g.C] = 0
    ss = raw.view(rows, -1, 16).pow(2).sum(-1).contiguous()
    w = rnd(g.H * (g.N + g.R), g.Q, seed=4, dtype=dtype, scale=g.Q ** -0.5)
    qn_w, kv_w = rnd(g.Q, seed=5), rnd(g.C, seed=6)
    pos = torch.randint(0, 300, (rows,), generator=torch.Generator().manual_seed(2)).to(torch.int32).to(DEV)
    slot = torch.randperm(128, generator=torch.Generator().manual_seed(3))[:rows].to(torch.int32).to(DEV)
    if rows > 2:
        slot[1] = -1                                              # an idle row stores nothing
    cache = torch.full((128, g.C + g.R), 5.0, dtype=dtype, device=DEV)
    xq = octets((raw[:, :g.Q] * qn_w).to(dtype))
    qn, q = ol.query_and_append(xq, raw, ss, ol.TileWeight(w), g, kv_w, eps, rope, pos, slot, cache)
    cq = f(ol.act_rows(xq)) / torch.sqrt(raw[:, :g.Q].pow(2).sum(-1, keepdim=True) / g.q_real + eps)
    full = (cq @ f(w).T).view(rows, g.H, g.N + g.R)
    torch.testing.assert_close(f(qn), full[..., :g.N], **OP[dtype])
    torch.testing.assert_close(f(q[..., g.C:]), rope.turn(full[..., g.N:], pos), **OP[dtype])
    c = raw[:, g.Q:g.Q + g.C]
    c = c / torch.sqrt(c.pow(2).sum(-1, keepdim=True) / g.c_real + eps) * kv_w
    line = torch.cat([c, rope.turn(raw[:, g.Q + g.C:g.Q + g.C + g.R], pos)], 1)
    keep = slot >= 0
    torch.testing.assert_close(f(cache[slot[keep].long()]), line[keep], **OP[dtype])
    rest = torch.ones(128, dtype=torch.bool, device=DEV)
    rest[slot[keep].long()] = False
    assert bool((cache[rest] == 5).all())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", ROWS)
def test_per_head_projections_and_gate(ol, dtype, rows):
    g = Geom(5, 64, 32, 96, 128, 32)
    uk, uv = rnd(g.H, g.C, g.N, seed=1, dtype=dtype, scale=0.1), rnd(g.H, g.V, g.C, seed=2, dtype=dtype, scale=0.1)
    qn, q = rnd(rows, g.H, g.N, seed=3, dtype=dtype), torch.full((rows, g.H, g.C + g.R), 3.0, dtype=dtype, device=DEV)
    ol.query_to_latent(qn, ol.TileWeight(uk), q, g)
    want = torch.stack([f(qn[:, h]) @ f(uk[h]).T for h in range(g.H)], 1)
    torch.testing.assert_close(f(q[..., :g.C]), want, **OP[dtype])
    assert bool((q[..., g.C:] == 3).all())
    o, raw = rnd(rows, g.H, g.C, seed=4, dtype=dtype), rnd(rows, 64 + g.H * g.V, seed=5)
    act = torch.full((rows, g.H * g.V + 32), 3.0, dtype=dtype, device=DEV)
    ol.latent_to_value(o, ol.TileWeight(uv), raw, 64, act, g)
    want = torch.stack([f(o[:, h]) @ f(uv[h]).T for h in range(g.H)], 1).reshape(rows, -1) * torch.sigmoid(raw[:, 64:])
    torch.testing.assert_close(f(act[:, :g.H * g.V]), want, **OP[dtype])
    assert bool((act[:, g.H * g.V:] == 3).all())
    block = torch.full((act.shape[1] // 8, rows, 8), 3.0, dtype=dtype, device=DEV)
    ol.latent_to_value(o, ol.TileWeight(uv), raw, 64, block, g)
    assert torch.equal(ol.act_rows(block), act)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", ROWS)
def test_residual_and_token_gemms(ol, dtype, rows):
    w, a, x = rnd(96, 160, seed=1, dtype=dtype), rnd(rows, 160, seed=2, dtype=dtype), rnd(rows, 96, seed=3)
    want, x2 = x + f(a) @ f(w).T, x.clone()
    ol.add_linear(a, ol.TileWeight(w), x)
    xt = ol.add_linear(octets(a), ol.TileWeight(w), x2, want_copy=True)
    assert torch.equal(x, x2) and torch.equal(ol.act_rows(xt), x.to(dtype))
    torch.testing.assert_close(x, want, atol=1e-3, rtol=1e-4)
    w, table = rnd(32, 96, seed=4, dtype=dtype, scale=0.1), rnd(50, 60, seed=5, dtype=dtype)
    ids = torch.randint(0, 50, (rows,), generator=torch.Generator().manual_seed(1)).to(DEV)
    part = table[:, 20:43]
    y = ol.token_gate_linear(xt, ol.TileWeight(w), part, ids, 23)
    assert torch.equal(ol.token_gate_linear(ol.act_rows(xt).contiguous(), ol.TileWeight(w), part, ids, 23), y)
    want = R.gelu((f(x.to(dtype)) @ f(w).T)[:, :23]) * f(part[ids])
    torch.testing.assert_close(f(y[:, :23]), want, **OP[dtype])
    assert bool((y[:, 23:] == 0).all())


# ---- row kernels ------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("real,width", [(40, 64), (1056, 1056), (5000, 5024)])
@pytest.mark.parametrize("parts", ["embed", "embed step", "y", "y step", "step", ""])
def test_finish(ol, dtype, real, width, parts):
    rows, eps = 3, 1e-2
    pad = lambda t: torch.nn.functional.pad(t, (0, width - real))
    x, nw, yw, step = pad(rnd(rows, real, seed=1)), pad(rnd(real, seed=2)), pad(rnd(real, seed=3)), pad(rnd(real, seed=4))
    emb, ids = pad(rnd(11, real, seed=5, dtype=dtype)), torch.tensor([10, 0, 3], device=DEV)
    for ydt in {torch.float32, dtype}:
        y = pad(rnd(rows, real, seed=6, dtype=ydt))
        want = f(emb[ids]) if "embed" in parts else x.clone()
        if "y" in parts:
            want = want + f(y) / torch.sqrt(f(y).pow(2).sum(-1, keepdim=True) / real + eps) * yw
        if "step" in parts:
            want = want + step
        got = x.clone()
        h = ol.finish(got, nw, eps, real, dtype, embed=emb if "embed" in parts else None, ids=ids if "embed" in parts else None,
                      y=y if "y" in parts else None, y_w=yw if "y" in parts else None, step=step if "step" in parts else None)
        torch.testing.assert_close(got, want, atol=1e-5, rtol=1e-5)
        h2 = ol.finish(got.clone(), nw, eps, real, dtype, octets=True)
        torch.testing.assert_close(f(ol.act_rows(h2)), f(h), atol=1e-6, rtol=1e-2)
        torch.testing.assert_close(f(h), want / torch.sqrt(want.pow(2).sum(-1, keepdim=True) / real + eps) * nw, **OP[dtype])


@pytest.mark.parametrize("dtype", DTYPES)
def test_prepare_residual_gather(ol, dtype):
    g = Geom(2, 32, 32, 32, 64, 96, c_real=50, q_real=70)
    rows, eps, n_up, up_off = 37, 1e-3, 40, 96 + 64 + 32 + 64
    rope = Rope(300, g.R // 2 - 2)
    y = rnd(rows, up_off + n_up, seed=1, dtype=dtype)
    y[:, g.q_real:g.Q] = 0
    y[:, g.Q + g.c_real:g.Q + g.C] = 0
    qw, kw = rnd(g.Q, seed=2), rnd(g.C, seed=3)
    pos = (torch.arange(rows) * 7).to(torch.int32).to(DEV)
    slot = torch.randperm(64, generator=torch.Generator().manual_seed(1))[:rows].to(torch.int32).to(DEV)
    cache = torch.full((64, g.C + g.R), 5.0, dtype=dtype, device=DEV)
    act = torch.full((rows, 64 + n_up), 7.0, dtype=dtype, device=DEV)
    cq, ck = ol.prepare(y, g, up_off, n_up, qw, kw, eps, rope, pos, slot, cache, act, 64, want_rows=True)
    yf = f(y)
    q = yf[:, :g.Q]
    torch.testing.assert_close(f(cq), q / torch.sqrt(q.pow(2).sum(-1, keepdim=True) / g.q_real + eps) * qw, **OP[dtype])
    c = yf[:, g.Q:g.Q + g.C]
    line = torch.cat([c / torch.sqrt(c.pow(2).sum(-1, keepdim=True) / g.c_real + eps) * kw,
                      rope.turn(yf[:, g.Q + g.C:g.Q + g.C + g.R], pos)], 1)
    torch.testing.assert_close(f(ck), line, **OP[dtype])
    assert torch.equal(ol.gather_rows(cache, slot), ck)
    torch.testing.assert_close(f(act[:, 64:]), R.gelu(yf[:, up_off:]), **OP[dtype])
    assert bool((act[:, :64] == 7).all())
    x, d = rnd(rows, 64, seed=4), rnd(rows, 64, seed=5, dtype=dtype)
    want = x + f(d)
    xt = ol.residual(d, x, True)
    assert torch.equal(x, want) and torch.equal(xt, want.to(dtype))
    table, ids = rnd(20, 48, seed=6, dtype=dtype), torch.arange(rows, device=DEV) % 20
    s = rnd(rows, 64, seed=7, dtype=dtype)
    out = ol.token_gate(s, table[:, 8:41], ids, 33)
    torch.testing.assert_close(f(out[:, :33]), R.gelu(f(s[:, :33])) * f(table[ids, 8:41]), **OP[dtype])
    assert bool((out[:, 33:] == 0).all())


def test_decode_prep(ol):
    i32 = lambda *v: torch.tensor(v, dtype=torch.int32, device=DEV)
    lens, table = i32(0, 63, 64, -1, 130, 192), torch.arange(18, dtype=torch.int32, device=DEV).view(6, 3).flip(1).contiguous()
    pos, slot, klen = i32(*[9] * 6), i32(*[9] * 6), i32(*[9] * 6)
    ol.decode_prep(lens, table, pos, slot, klen)
    assert pos.tolist() == [0, 63, 64, 0, 130, 0] and klen.tolist() == [1, 64, 65, 0, 131, 0]
    assert slot.tolist() == [2 * 64, 5 * 64 + 63, 7 * 64, -1, 12 * 64 + 2, -1]
    assert lens.tolist() == [1, 64, 65, -1, 131, 192], "rows that are idle or past their table stay where they are"


# ---- attention --------------------------------------------------------------------------------------------------------------
BORDERS = [1, 15, 16, 17, 63, 64, 65, 127, 128, 129, 300]


def _paged(lens, C, Rr, dtype, seed, extra=3):
    """Pages in shuffled order; whatever no sequence has written is NaN."""
    need = [-(-n // 64) for n in lens]
    n_pages = sum(need) + extra
    order = torch.randperm(n_pages, generator=torch.Generator().manual_seed(seed)).tolist()
    cache = torch.full((n_pages * 64, C + Rr), float("nan"), dtype=dtype, device=DEV)
    table = torch.zeros(len(lens), max(need + [1]) + 1, dtype=torch.int32)
    keys = []
    for b, n in enumerate(lens):
        k = rnd(n, C + Rr, seed=seed + 10 + b, dtype=dtype)
        for p in range(need[b]):
            table[b, p] = order.pop()
            part = k[p * 64:(p + 1) * 64]
            cache[int(table[b, p]) * 64:int(table[b, p]) * 64 + len(part)] = part
        keys.append(k)
    return cache, table.to(DEV), keys


DEC_SHAPES = [(1, 32, 32), (4, 64, 32), (16, 128, 32), (20, 96, 64), (40, 160, 32), (20, 512, 64), (16, 512, 64), (3, 320, 64)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("nsplit", [1, 2, 7, 256])
@pytest.mark.parametrize("heads,C,Rr", DEC_SHAPES)
def test_attn_decode(ol, dtype, heads, C, Rr, nsplit):
    lens = BORDERS + [0]
    cache, table, keys = _paged(lens, C, Rr, dtype, 5)
    q = rnd(len(lens), heads, C + Rr, seed=1, dtype=dtype)
    klen = torch.tensor(lens, dtype=torch.int32, device=DEV)
    scale = 1.5 * (C + Rr) ** -0.5
    out = f(ol.attn_decode(q, cache, table, klen, Geom(heads, 32, Rr, 32, C, 32), scale, max(lens), nsplit=nsplit))
    for b, n in enumerate(lens):
        if n == 0:
            assert bool((out[b] == 0).all())
            continue
        k = f(keys[b])
        want = torch.softmax(f(q[b]) @ k.T * scale, -1) @ k[:, :C]
        torch.testing.assert_close(out[b], want, **(dict(atol=2e-5, rtol=2e-5) if dtype == torch.float32 else dict(atol=1e-2, rtol=1e-2)))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,C,Rr", [(4, 64, 32), (20, 512, 64)])
def test_attn_decode_finds_one_key_anywhere(ol, dtype, heads, C, Rr):
    """One key matches the query and takes nearly all the weight: at the first token, at page borders, at the last one; the row
    right behind the last (NaN) must not count."""
    n = 200
    spots = [0, 1, 62, 63, 64, 65, 127, 128, 191, 192, 199]
    cache, table, keys = _paged([n] * len(spots), C, Rr, dtype, 9)
    q = torch.stack([keys[b][s].expand(heads, -1) for b, s in enumerate(spots)]).contiguous()
    klen = torch.full((len(spots),), n, dtype=torch.int32, device=DEV)
    for nsplit in (1, 3):
        out = f(ol.attn_decode(q, cache, table, klen, Geom(heads, 32, Rr, 32, C, 32), 1.0, n, nsplit=nsplit))
        for b, s in enumerate(spots):
            torch.testing.assert_close(out[b], f(keys[b][s, :C]).expand(heads, -1), atol=1e-2, rtol=1e-2)


PRE_SHAPES = [(2, 32, 32, 32, 32), (3, 64, 32, 64, 96), (2, 128, 64, 128, 512), (2, 160, 64, 224, 320), (1, 320, 64, 256, 64), (64, 128, 64, 128, 64)]


def _prefill_case(g, news, pasts, dtype, seed):
    seq, at_q, at_k = [], 0, 0
    for n, p in zip(news, pasts):
        seq.append((at_q, n, at_k, n + p))
        at_q, at_k = at_q + n, at_k + n + p
    q = rnd(at_q, g.H * (g.N + g.R), seed=seed, dtype=dtype)
    kv = rnd(at_k, g.H * (g.N + g.V), seed=seed + 1, dtype=dtype)
    ck = rnd(at_k, g.C + g.R, seed=seed + 2, dtype=dtype)
    pos = torch.cat([torch.arange(p, p + n) for n, p in zip(news, pasts)]).to(torch.int32).to(DEV)
    return q, kv, ck, torch.tensor(seq, dtype=torch.int32, device=DEV), pos


def _prefill_want(g, q, kv, ck, seq, pos, rope, gate, scale):
    out = []
    for qa, n, ka, nk in seq.tolist():
        qq = f(q[qa:qa + n]).view(n, g.H, g.N + g.R)
        qr = rope.turn(qq[..., g.N:], pos[qa:qa + n])
        kk = f(kv[ka:ka + nk])
        kn, v = kk[:, :g.H * g.N].view(nk, g.H, g.N), kk[:, g.H * g.N:].view(nk, g.H, g.V)
        kr = f(ck[ka:ka + nk, g.C:])
        s = torch.stack([qq[:, h, :g.N] @ kn[:, h].T + qr[:, h] @ kr.T for h in range(g.H)]) * scale
        hide = torch.arange(nk, device=DEV)[None, :] > torch.arange(nk - n, nk, device=DEV)[:, None]
        p = torch.softmax(s.masked_fill(hide, float("-inf")), -1)
        out.append(torch.stack([p[h] @ v[:, h] for h in range(g.H)], 1).reshape(n, -1))
    return torch.cat(out) * torch.sigmoid(f(gate))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,N,Rr,V,C", PRE_SHAPES)
@pytest.mark.parametrize("news,pasts", [((1,), (0,)), ((2, 1, 63, 65), (0, 0, 0, 0)), ((130, 5, 64), (0, 190, 64)), ((300,), (1,)), ((520, 300), (0, 77))])
def test_attn_prefill(ol, dtype, heads, N, Rr, V, C, news, pasts):
    g = Geom(heads, N, Rr, V, C, 32)
    q, kv, ck, seq, pos = _prefill_case(g, news, pasts, dtype, 3)
    rope = Rope(700, Rr // 2)
    tq = q.shape[0]
    gate = rnd(tq, g.H * g.V, seed=8, dtype=dtype)
    act = torch.full((tq, g.H * g.V + 32), 3.0, dtype=dtype, device=DEV)
    scale = 1.5 * (N + Rr) ** -0.5
    ol.attn_prefill(q, kv, ck, seq, max(news), pos, rope, gate, act, g, scale)
    if dtype == torch.bfloat16:                                   # the rotated query is an operand: rounded like the kernel's
        qv = q.view(tq, g.H, N + Rr).clone()
        qv[..., N:] = rope.turn(f(qv[..., N:]), pos).to(dtype)
        want = _prefill_want(g, qv.view(tq, -1), kv, ck, seq, torch.zeros_like(pos), _NoRope(), gate, scale)
    else:
        want = _prefill_want(g, q, kv, ck, seq, pos, rope, gate, scale)
    torch.testing.assert_close(f(act[:, :g.H * g.V]), want, **(dict(atol=3e-5, rtol=3e-5) if dtype == torch.float32 else dict(atol=2e-2, rtol=2e-2)))
    assert bool((act[:, g.H * g.V:] == 3).all())


class _NoRope:
    def turn(self, x, pos):
        return x


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,N,Rr,V,C", [(2, 32, 32, 32, 32), (2, 128, 64, 128, 512)])
def test_attn_prefill_finds_one_key_and_not_the_next(ol, dtype, heads, N, Rr, V, C):
    """Query j looks for key s: found when s <= j, and the key right behind a query (s = j + 1) stays invisible."""
    g, n, past = Geom(heads, N, Rr, V, C, 32), 260, 70
    rope = Rope(400, Rr // 2)
    q, kv, ck, seq, pos = _prefill_case(g, (n,), (past,), dtype, 3)
    gate = torch.full((n, g.H * g.V), 60.0, dtype=dtype, device=DEV)                     # sigmoid = 1
    pairs = [(0, 0), (0, past), (63, 5), (64, past + 63), (65, 64), (127, past + 127), (128, 127), (130, 128), (200, past + 1),
             (259, past + 259), (259, 0), (191, past + 190)]
    hidden = [(10, past + 11), (63, past + 64), (126, past + 127), (127, past + 128)]
    kn = kv[:, :g.H * N].view(-1, g.H, N)
    qv = q.view(n, g.H, N + Rr)
    qv[..., N:] = 0
    v = f(kv[:, g.H * N:])
    for j, s in pairs + hidden:
        qv[j, :, :N] = kn[s]
        out = torch.empty(n, g.H * g.V, dtype=dtype, device=DEV)
        ol.attn_prefill(q, kv, ck, seq, n, pos, rope, gate, out, g, 2.0)
        found = bool(((f(out[j]) - v[s]).abs() < 5e-2).float().mean() > 0.98)
        assert found == ((j, s) in pairs), (j, s)


# ---- whole models -----------------------------------------------------------------------------------------------------------
def build(cfg, sd, dtype, budget=900, batch=6, graphs=True):
    from triforce_amd.models.cache import LatentCache
    from triforce_amd.models.config_befidra import BefidraConfig
    from triforce_amd.models.modeling_befidra import BefidraForCausalLM
    from triforce_amd.utils.batch_infer import BatchInferenceEngine
    m = BefidraForCausalLM.from_state_dict(BefidraConfig.from_dict(cfg), sd, DEV, dtype)
    return BatchInferenceEngine(m, LatentCache(m, budget, batch), use_graphs=graphs)


@pytest.fixture(scope="module")
def models():
    made = {}

    def get(name, dtype):
        if (name, dtype) not in made:
            cfg = H.CONFIGS[name]
            sd = H.weights(cfg, 11, sharp=2.5 if dtype == torch.float32 else 1.0)
            made[name, dtype] = (cfg, sd, build(cfg, sd, dtype))
        cfg, sd, e = made[name, dtype]
        e.clear_kv()
        return cfg, sd, e
    yield get
    made.clear()                                                  # captured graphs go with their engines


def feed(e, name, toks, cuts):
    """Portions of the given sizes, then the rest token by token -> logits of every position."""
    out, at = [], 0
    for n in list(cuts) + [1] * (len(toks) - sum(cuts)):
        out.append(e.step([(name, toks[at:at + n], range(n))]).clone())
        at += n
    return torch.cat(out)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(H.CONFIGS))
def test_model_whole_portions_and_decode(models, name, dtype):
    cfg, sd, e = models(name, dtype)
    toks = H.tokens_of(cfg, 150, 3)
    want, tol = H.oracle_logits(cfg, sd, toks), H.bound(cfg, sd, toks, dtype)
    for cuts in ([150], [2] * 5 + [1, 60, 79], [64, 64, 22], [63, 2, 85], [1], [140]):
        got = feed(e, "s", toks, cuts)
        err = H.error(got, want)
        print(f"[latent] {name} {dtype} cuts {cuts[:4]}: {err:.2e} of {tol:.2e}", flush=True)
        assert err < tol, (cuts, err, tol)
        e.kv_cache.release("s")


def test_residual_after_every_layer_run(models):
    cfg, sd, e = models("mixed", torch.float32)
    toks, want = H.tokens_of(cfg, 40, 9), []
    R.forward(cfg, {k: v.double() for k, v in sd.items()}, toks, want)
    e.model.weights.capture = got = []
    try:
        e.step([("s", toks, range(40))])
    finally:
        e.model.weights.capture = None
    assert len(want) == len(got) == 7
    for a, b in zip(got, want):
        torch.testing.assert_close(a.cpu(), b.float(), atol=2e-4, rtol=1e-4)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "wide", "once"])
def test_batches_of_unequal_requests_against_each_alone(models, name, dtype):
    """Prefilled together, decoded in lockstep, shorter ones leave; their pages are used by the next batch."""
    cfg, sd, e = models(name, dtype)
    c = e.kv_cache
    for rnd_no, sizes in enumerate([(1, 70, 130, 64, 5), (129, 2, 63), (40,) * 6]):
        toks = [H.tokens_of(cfg, n + 12 - i, 100 * rnd_no + i) for i, n in enumerate(sizes)]
        got = [[] for _ in sizes]
        out = e.step([(i, t[:n], [n - 1]) for i, (n, t) in enumerate(zip(sizes, toks))]).clone()
        for i in range(len(sizes)):
            got[i].append(out[i:i + 1])
        live = list(range(len(sizes)))
        at = list(sizes)
        while live:
            out = e.step([(i, toks[i][at[i]:at[i] + 1], [0]) for i in live], [i for i in live if at[i] + 1 == len(toks[i])]).clone()
            for b, i in enumerate(live):
                got[i].append(out[b:b + 1])
                at[i] += 1
            live = [i for i in live if at[i] < len(toks[i])]
        assert c.tokens == 0 and len(c.free) == c.n_pages
        for i, n in enumerate(sizes):
            want = H.oracle_logits(cfg, sd, toks[i])[n - 1:]
            assert H.error(torch.cat(got[i]), want) < H.bound(cfg, sd, toks[i], dtype), (sizes, i)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_and_freed_pages(models, dtype):
    """Two sequences advance over many page borders while a third comes and goes in between (its pages change owners)."""
    cfg, sd, e = models("mixed", dtype)
    a, b, x = H.tokens_of(cfg, 330, 1), H.tokens_of(cfg, 290, 2), H.tokens_of(cfg, 90, 3)
    got_a, got_b = [e.step([("a", a[:50], [49])]).clone()], [e.step([("b", b[:10], [9])]).clone()]
    for n in range(280):
        if n % 70 == 5:
            e.step([("x", x, [])])
        if n % 70 == 40:
            e.step([], ["x"])
        out = e.step([("a", [a[50 + n]], [0]), ("b", [b[10 + n]], [0])]).clone()
        got_a.append(out[:1])
        got_b.append(out[1:])
    assert H.error(torch.cat(got_a), H.oracle_logits(cfg, sd, a)[49:]) < H.bound(cfg, sd, a, dtype)
    assert H.error(torch.cat(got_b), H.oracle_logits(cfg, sd, b)[9:]) < H.bound(cfg, sd, b, dtype)


def test_mixed_portions_of_many_sequences(models):
    """Portions of one step have different pasts, one of them none."""
    cfg, sd, e = models("mixed", torch.float32)
    toks = [H.tokens_of(cfg, 120, 20 + i) for i in range(3)]
    e.step([(0, toks[0][:70], []), (1, toks[1][:1], [])])
    out = e.step([(1, toks[1][1:3], [0, 1]), (2, toks[2][:64], [63]), (0, toks[0][70:], [0, 49])])
    want = [H.oracle_logits(cfg, sd, t) for t in toks]
    assert H.error(out, torch.stack([want[1][1], want[1][2], want[2][63], want[0][70], want[0][119]])) < F32


def test_prompt_longer_than_a_forward(models, monkeypatch):
    from triforce_amd.utils import graph_infer
    monkeypatch.setattr(graph_infer, "PREFILL_CHUNK", 128)
    cfg, sd, e = models("mixed", torch.float32)
    toks = [H.tokens_of(cfg, n, n) for n in (300, 90)]
    out = e.step([(0, toks[0], [299, 0, 128, 127]), (1, toks[1], [89])])
    w0, w1 = (H.oracle_logits(cfg, sd, t) for t in toks)
    assert H.error(out, torch.stack([w0[299], w0[0], w0[128], w0[127], w1[89]])) < F32


@pytest.mark.parametrize("dtype", DTYPES)
def test_graph_replays_equal_eager_steps(dtype):
    """The captured decode step against the eager one, bit for bit, over replays with changing batches in between."""
    cfg = H.CONFIGS["mixed"]
    sd = H.weights(cfg, 21)
    eager, graph = build(cfg, sd, dtype, graphs=False), build(cfg, sd, dtype, graphs=True)
    toks = [H.tokens_of(cfg, 90, 40 + i) for i in range(3)]
    for e in (eager, graph):
        e.step([(i, t[:20 + 22 * i], []) for i, t in enumerate(toks)])
    for n in range(25):
        who = [0, 1, 2] if n % 5 else [2, 0]
        for r in range(1 if n % 3 else 2):
            entries = [(i, [toks[i][(n + r) % 90]], [0]) for i in who]
            a, b = eager.step(entries).clone(), graph.step(entries).clone()
            torch.cuda.synchronize()
            assert torch.equal(a, b), n


def test_refused_steps_leave_everything_as_it_was(models):
    cfg, sd, e = models("plain", torch.float32)
    e.step([("a", [1, 2, 3], [])])
    for bad, exc in (([("a", [1], [0]), ("a", [2], [0])], ValueError), ([("a", [], [])], ValueError), ([("a", [1], [1])], ValueError),
                     ([("a", [cfg["vocab"]], [0])], ValueError), ([("a", [1], [0]), ("b", [1] * 899, [])], IndexError)):
        with pytest.raises(exc):
            e.step(bad)
    with pytest.raises(KeyError):
        e.step([("a", [1], [0])], ["nobody"])
    out = e.step([("a", [4], [0])])
    assert H.error(out, H.oracle_logits(cfg, sd, [1, 2, 3, 4])[3:]) < F32


# ---- the framework's entry points -------------------------------------------------------------------------------------------
def greedy_oracle(cfg, sd, prompt, n):
    sd = {k: v.double() for k, v in sd.items()}
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(R.forward(cfg, sd, toks)[-1].argmax()))
    return toks[len(prompt):]


def test_greedy_generation_batched_and_single(models):
    from triforce_amd.utils.decoding import Autoregressive, AutoregressiveBatch
    from triforce_amd.utils.sampling import UniformSource
    cfg, sd, _ = models("mixed", torch.float32)
    e = build(cfg, sd, torch.float32, budget=170, batch=3)       # four prompts: not all of them fit at once
    prompts = [H.tokens_of(cfg, n, 60 + n) for n in (5, 66, 30, 61)]
    lens = [9, 4, 12, 6]
    want = [greedy_oracle(cfg, sd, p, n + 1) for p, n in zip(prompts, lens)]
    kw = dict(temperature=1.0, top_p=1e-9, rng=UniformSource(DEV, seed=1), return_tokens=True)
    speed, got = AutoregressiveBatch(None, e, prompts, max_len=lens, **kw)
    assert got == want and speed > 0
    assert e.kv_cache.tokens == 0
    _, ids = Autoregressive(None, e, torch.tensor([prompts[1]], device=DEV), max_len=lens[1], **kw)
    assert ids == want[1]
    with pytest.raises(IndexError):
        AutoregressiveBatch(None, e, [prompts[0]], max_len=400, **kw)


def test_generate_script(capsys, monkeypatch):
    import importlib.util
    import os
    path = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "test", "generate.py")
    spec = importlib.util.spec_from_file_location("generate_script", path)
    mod = importlib.util.module_from_spec(spec)
    spec.loader.exec_module(mod)
    mod.main(["--target", "befidra-tiny", "--batch", "3", "--prefill", "90", "--gen_len", "12", "--greedy"])
    text = capsys.readouterr().out
    assert "prompt 90 tokens" in text and "tokens/s" in text


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_from_a_checkpoint_directory(tmp_path, dtype):
    """config.json + model.safetensors -> registry -> engine -> files of logits."""
    from safetensors.torch import save_file
    from triforce_amd.utils import trace
    cfg = H.CONFIGS["loop_all"]
    sd = H.weights(cfg, 31, sharp=1.0)
    (tmp_path / "model").mkdir()
    (tmp_path / "out").mkdir()
    (tmp_path / "model" / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in sd.items()}, str(tmp_path / "model" / "model.safetensors"))
    e = trace.make_engine(trace.parse(["--model", str(tmp_path / "model"), "--out", str(tmp_path / "out"), "--max-tokens", "120",
                                       "--dtype", dtype]))
    a, b = H.tokens_of(cfg, 70, 1), H.tokens_of(cfg, 40, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:66], "want": [65, 3]}, {"id": "b", "tokens": b[:39], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[66:67], "want": []}, {"id": "b", "tokens": b[39:], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[67:68], "want": [0]}], "end": ["a"]}]
    seen = []
    trace.replay(e, [json.dumps(s) for s in steps], str(tmp_path / "out"), seen.append)
    assert seen == ["done 0", "done 1", "done 2"]
    wa, wb = H.oracle_logits(cfg, sd, a), H.oracle_logits(cfg, sd, b)
    read = lambda n: torch.frombuffer(bytearray((tmp_path / "out" / f"{n}.f32").read_bytes()), dtype=torch.float32).view(-1, cfg["vocab"])
    tol = H.bound(cfg, sd, a, getattr(torch, dtype))
    assert H.error(read(0), torch.stack([wa[65], wa[3]])) < tol
    assert H.error(read(1), wb[39:]) < tol and H.error(read(2), wa[67:68]) < tol
