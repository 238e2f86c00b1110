"""Small Befidra configurations and weights of the latent tests (device side and oracle/ref_latent.py from the same tensors)."""
import torch

from oracle import ref_latent as R


def mixer(heads, dim, rot_dim, vdim, q_rank, kv_rank, base=10000.0, yarn=None, scale=None):
    scaling = None if yarn is None else dict(zip(("factor", "original", "fast", "slow"), yarn))
    return dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank,
                scale=scale if scale is not None else (dim + rot_dim) ** -0.5, rot=dict(dims=rot_dim, base=base, scaling=scaling))


def config(vocab, width, layers, eps=1e-5, loop=None, side=None):
    d = dict(architecture="Befidra", vocab=vocab, width=width, norm=dict(eps=eps),
             layers=[dict(type="latent_attention", mixer=m, mlp=None if ff is None else dict(kind="dense", ff=ff)) for m, ff in layers])
    if loop is not None:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    if side is not None:
        d["token_side"] = dict(dim=side)
    return d


CONFIGS = {
    # every layer its own sizes, one layer without a feed-forward, a loop in the middle that runs three times
    "mixed": config(131, 88, [(mixer(2, 24, 8, 40, 20, 36, yarn=(4.0, 64, 8.0, 1.0)), 72),
                              (mixer(5, 32, 16, 24, 48, 64, base=500.0, yarn=(2.0, 32, 4.0, 0.5)), None),
                              (mixer(3, 16, 12, 56, 33, 40, base=100.0, scale=0.25), 50)], eps=1e-3, loop=(1, 3, 3), side=10),
    # one head, the smallest rotation, no loop, no token side
    "plain": config(67, 40, [(mixer(1, 10, 2, 6, 7, 9), 30), (mixer(1, 33, 4, 65, 31, 65, base=50.0), 1)]),
    # the whole stack looped; loop of a single pass is "once"
    "loop_all": config(97, 64, [(mixer(4, 32, 32, 32, 32, 32, yarn=(8.0, 16, 2.0, 0.25)), 64)] * 2, loop=(0, 2, 2), side=32),
    "once": config(97, 64, [(mixer(2, 16, 8, 16, 24, 24), 40)] * 2, loop=(1, 2, 1), side=1),
    # the specialised shapes: 512 + 64 rows, 128 + 64 / 128 heads; more heads than one tile, more than one head group
    "wide": config(80, 96, [(mixer(20, 128, 64, 128, 64, 512, yarn=(16.0, 64, 8.0, 1.0)), 96)] * 2, side=16),
    "groups": config(80, 96, [(mixer(33, 16, 16, 16, 40, 48), 96), (mixer(3, 160, 64, 200, 64, 300), None)], loop=(0, 1, 2)),
}


def weights(cfg, seed, sharp=2.5):
    """Random weights with attention that is far from flat (``sharp`` = mean query norm weight: 2.5 makes single keys stand out,
    which in bfloat16 also magnifies rounding - those tests take 1), norms away from 1, and every value representable in bfloat16
    (both sides then start from the same numbers)."""
    g = torch.Generator().manual_seed(seed)
    from triforce_amd.models.config_befidra import BefidraConfig
    from triforce_amd.models.latent_core import LatentWeights
    shapes = LatentWeights(BefidraConfig.from_dict(cfg), "cpu", torch.float32).shapes()
    sd = {}
    for n, s in shapes.items():
        r = torch.randn(s, generator=g)
        if n.endswith("mix.dq.norm"):
            w = sharp + 0.2 * sharp * r
        elif n.endswith("norm") or n.endswith("norm1"):
            w = 1.0 + 0.3 * r
        elif n == "embed" or n == "loop.step":
            w = r
        elif n == "side.embed":
            w = 2.0 * r
        else:
            w = 1.5 * r * s[1] ** -0.5
        sd[n] = w.to(torch.bfloat16).to(torch.float32)
    return sd


def oracle_logits(cfg, sd, tokens):
    return R.forward(cfg, {k: v.double() for k, v in sd.items()}, tokens).float()


def bound(cfg, sd, tokens, dtype):
    """What ``error`` may be: a fixed bound in float32; in bfloat16 three times what rounding the operands of every matrix product
    does to the oracle itself."""
    if dtype == torch.float32:
        return 5e-5
    sd = {k: v.double() for k, v in sd.items()}
    rounded = R.forward(cfg, sd, tokens, operand=lambda x: x.to(torch.bfloat16).double())
    return 3 * error(rounded, R.forward(cfg, sd, tokens))


def tokens_of(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def error(got, want):
    """Root mean square difference of logit rows over the spread of the expected logits: worst row."""
    got, want = got.float().cpu(), want.float().cpu()
    d = (got - want).pow(2).mean(-1).sqrt()
    return float((d / want.std()).max())
